"""Trace runner: feeds given token ids through a model, step by step, and writes logits.

    bin/trace_run --model DIR --dtype bfloat16|float32 --out DIR --max-tokens N

Steps come from standard input, one JSON object a line:

    {"step": 0, "entries": [{"id": "a", "tokens": [5, 17, 3], "want": [0, 2]}], "end": []}

Every step is one mixed batch of the engine (Engine.step): portions of prompts beside single tokens, from
the cache earlier steps left.  The logits at the wanted places go to OUT/<step>.f32 (little-endian fp32,
[wanted, vocab]); `done <step>` is printed after every step.  Requests in `end` give their slot and cache
blocks back.  --max-tokens sizes the cache pool.
"""
from __future__ import annotations

import argparse
import json
import os
import sys
from typing import Dict, List

import numpy as np

from ..models import registry
from . import native
from .loader import load_engine

MAX_LIVE = 4


class Replay:
    """Requests by id -> engine slots and positions."""

    def __init__(self, engine, slots: int):
        self.engine = engine
        self.free = list(range(slots))
        self.live: Dict[str, List[int]] = {}  # id -> [slot, position]

    def step(self, entries: list, end: list) -> np.ndarray:
        slots, starts, counts, tokens, want = [], [], [], [], []
        for e in entries:
            if e["id"] not in self.live:
                if not self.free:
                    raise RuntimeError("more live requests than slots")
                self.live[e["id"]] = [self.free.pop(), 0]
            r, ids = self.live[e["id"]], [int(t) for t in e["tokens"]]
            if not ids:
                continue
            slots.append(r[0])
            starts.append(r[1])
            counts.append(len(ids))
            want.extend(len(tokens) + int(w) for w in e.get("want", []))
            tokens.extend(ids)
            r[1] += len(ids)
        out = np.zeros((0, 0), np.float32)
        if slots:
            rows = sorted(set(want))  # (the engine takes them ascending)
            out = self.engine.step(slots, starts, counts, tokens, rows)
            if rows != want:
                out = out[[rows.index(w) for w in want]]
        for i in end:
            if i in self.live:
                slot, _ = self.live.pop(i)
                self.engine.release_slot(slot)
                self.free.append(slot)
        return out


def main(argv=None) -> int:
    ap = argparse.ArgumentParser(prog="trace_run", description="replay a trace of token ids through a model")
    ap.add_argument("--model", required=True, help="folder with config.json and model.safetensors")
    ap.add_argument("--dtype", choices=("bfloat16", "float32"), default="bfloat16")
    ap.add_argument("--out", required=True, help="folder for the logits, <step>.f32")
    ap.add_argument("--max-tokens", type=int, required=True, help="tokens the cache pool holds")
    args = ap.parse_args(argv)
    cfg, _, _ = registry.load_config(args.model)
    native.require("bf16")
    ctx = cfg.max_ctx if cfg.learned_pos else args.max_tokens
    eng, _, _ = load_engine(args.model, max_ctx=ctx, max_slots=MAX_LIVE, max_batch=MAX_LIVE, compute=args.dtype,
                            kv_pool_tokens=args.max_tokens)
    replay = Replay(eng, MAX_LIVE)
    for line in sys.stdin:
        if not line.strip():
            continue
        s = json.loads(line)
        out = replay.step(s["entries"], s.get("end", []))
        if any(e.get("want") for e in s["entries"]):
            np.ascontiguousarray(out, dtype="<f4").tofile(os.path.join(args.out, f"{s['step']}.f32"))
        print(f"done {s['step']}", flush=True)
    return 0


if __name__ == "__main__":
    sys.exit(main())
