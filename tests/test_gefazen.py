"""Gefazen on the CPU: configuration, registry, checkpoint reader, trace replay bookkeeping, the scheduler's
mixed steps and limited cache pool (fake engine), and the oracle the GPU tests compare against -- including
that each mechanism, left out or shifted by one, would show in the logits those tests look at."""
import asyncio
import json
import math
import threading

import numpy as np
import pytest
import torch

import gefazen_oracle as O
from aios_amd.models import registry
from aios_amd.models.config import LayerConfig, get_preset
from aios_amd.runtime import safetensors
from aios_amd.runtime.scheduler import GenRequest, Scheduler
from aios_amd.runtime.trace import Replay


def rel(a, b):
    d = (a - b).double()
    d = d - d.mean(-1, keepdim=True)
    return float((d.pow(2).mean(-1).sqrt() / b.double().std(-1)).max())


def write_model(path, cfg, w):
    path.mkdir(parents=True, exist_ok=True)
    (path / "config.json").write_text(json.dumps(cfg))
    safetensors.write(str(path / "model.safetensors"),
                      {k: ("BF16", tuple(v.shape), v.contiguous().view(torch.int16).numpy().tobytes()) for k, v in w.items()})
    return str(path)


MIXED = O.make_config(layers=[O.make_layer(), O.make_layer(heads=5, dim=40, vdim=16, kv_rank=72, scale=0.31, ff=None),
                              O.make_layer(weights_of=0),
                              O.make_layer(heads=5, dim=40, vdim=16, kv_rank=72, scale=0.31, ff=None, weights_of=1)])


# ---- configuration and checkpoints -----------------------------------------------------------------
def test_config_reads_every_size_and_branch(tmp_path):
    path = write_model(tmp_path / "m", MIXED, O.random_weights(MIXED))
    cfg, raw, arch = registry.load_config(path)
    assert (cfg.vocab_size, cfg.d_model, cfg.max_ctx, cfg.norm_eps, cfg.n_layers) == (211, 96, 512, 3e-5, 4)
    assert cfg.layers[0] == LayerConfig(heads=3, dim=24, vdim=40, kv_rank=56, scale=0.17, ff=72)
    assert cfg.layers[1].ff == 0 and cfg.layers[1].weights_of == -1 and cfg.layers[3].weights_of == 1
    names = arch.tensor_names(raw)
    assert set(names) == set(O.tensor_shapes(MIXED)) and len(set(names.values())) == len(names)
    assert names["l1.mix.uk"] == "blk.1.attn_k_b.weight" and "l1.mlp.up" not in names and "l2.mix.q" not in names
    assert registry.is_checkpoint_dir(path) and not registry.is_checkpoint_dir(str(tmp_path))
    assert cfg.n_params() == pytest.approx(sum(math.prod(s) for s in O.tensor_shapes(MIXED).values()), rel=0.02)


@pytest.mark.parametrize("change, message", [
    (dict(type="other"), "mixer type"), (dict(mlp={"kind": "sparse", "ff": 8}), "feed-forward"),
    (dict(weights_of=7), "weights_of"), (dict(weights_of=0), "weights_of")])
def test_config_rejects_what_the_design_does_not_have(change, message):
    raw = O.make_config(layers=[dict(O.make_layer(), **change)])
    with pytest.raises(ValueError, match=message):
        registry.get("Gefazen").parse(raw, "m")


def test_unknown_architecture():
    with pytest.raises(ValueError, match="unknown model architecture"):
        registry.get("nothing")


def test_safetensors_reader_round_trip_and_bounds(tmp_path):
    p = str(tmp_path / "x.safetensors")
    a = np.arange(6, dtype=np.float32)
    safetensors.write(p, {"a": ("F32", (2, 3), a.tobytes()), "b": ("I32", (1,), np.int32(7).tobytes())})
    r = safetensors.SafetensorsReader(p)
    assert r.tensors["a"].shape == (2, 3) and (r.raw("a").view(np.float32) == a).all()
    assert r.raw("b").view(np.int32)[0] == 7
    data = open(p, "rb").read()
    for bad in (data[:4], data[:-4], (10 ** 9).to_bytes(8, "little") + data[8:]):
        open(p, "wb").write(bad)
        with pytest.raises(ValueError):
            safetensors.SafetensorsReader(p)


def test_presets_name_the_design():
    for name in ("gefazen-1b", "gefazen-7b", "test-gefazen"):
        cfg = get_preset(name)
        assert cfg.arch == "gefazen" and len(cfg.layers) == cfg.n_layers and cfg.n_params() > 0


# ---- oracle ----------------------------------------------------------------------------------------
def test_oracle_mechanisms_by_hand():
    x = torch.tensor([[3.0, -4.0]], dtype=O.DT)
    assert torch.allclose(O.rms_norm(x, torch.tensor([1.0, 2.0], dtype=O.DT), 0.5), x / math.sqrt(13.0) * torch.tensor([1.0, 2.0]))
    z = torch.linspace(-3, 3, 7, dtype=O.DT)
    assert torch.allclose(O.gelu_tanh(z), torch.nn.functional.gelu(z, approximate="tanh"))
    p = O.sink_softmax(torch.tensor([0.0, math.log(2.0)], dtype=O.DT), math.log(5.0))
    assert torch.allclose(p, torch.tensor([1 / 8, 2 / 8], dtype=O.DT))
    assert O.owner([{}, {"weights_of": 2}, {"weights_of": 0}], 1) == 0
    cfg = O.make_config(layers=[O.make_layer()])
    w = O.random_weights(cfg, 3)
    ids = [int(t) for t in np.random.default_rng(0).integers(0, 211, 20)]
    assert torch.allclose(O.forward(cfg, w, ids)[:9], O.forward(cfg, w, ids[:9]))  # causal


@pytest.mark.parametrize("fault", ["no sink", "no gate", "no position", "position off by one", "one key short",
                                   "sequential layer", "silu", "no latent norm", "own weights", "scale"])
def test_a_fault_in_any_mechanism_shows(fault, monkeypatch):
    """Planted in the oracle: the logits move by far more than the GPU tests' tolerances (3e-2 in bf16)."""
    cfg = MIXED
    w = O.random_weights(cfg, 1, qk_gain=2.0)
    ids = [int(t) for t in np.random.default_rng(1).integers(0, 211, 40)]
    good = O.forward(cfg, w, ids)
    if fault == "no sink":
        w = {k: (v - 100 if k.endswith(".sink") else v) for k, v in w.items()}
    elif fault == "no position":
        w = dict(w, pos=torch.zeros_like(w["pos"]))
    elif fault == "position off by one":
        w = dict(w, pos=w["pos"].roll(1, 0))
    elif fault == "silu":
        monkeypatch.setattr(O, "gelu_tanh", torch.nn.functional.silu)
    elif fault == "no latent norm":
        monkeypatch.setattr(O, "latent", lambda h, w, p, eps: h @ w[p + "dkv"].T * w[p + "dkv.norm"])
    elif fault == "scale":
        cfg = dict(cfg, layers=[dict(l, mixer=dict(l["mixer"], scale=0.125)) for l in cfg["layers"]])
    elif fault == "own weights":
        cfg = dict(cfg, layers=[dict(l, weights_of=0) if i == 2 else l for i, l in enumerate(cfg["layers"])])
        other = O.random_weights(dict(cfg, layers=[cfg["layers"][1]]), 9)
        w = dict(w, **{k.replace("l0.", "l1."): v for k, v in other.items() if k.startswith("l0.")})
    elif fault == "no gate":
        monkeypatch.setattr(O.torch, "sigmoid", lambda z: torch.ones_like(z))
    elif fault == "one key short":
        real = O.sink_softmax
        monkeypatch.setattr(O, "sink_softmax", lambda a, s: real(torch.cat([a[:-1], a[-1:] - 1e4]) if len(a) > 1 else a, s))
    elif fault == "sequential layer":
        real = O.gated_mlp
        monkeypatch.setattr(O, "gated_mlp", lambda h, w, p: real(h * 0.9, w, p))
    assert rel(O.forward(cfg, w, ids), good) > 0.06


# ---- trace replay bookkeeping ------------------------------------------------------------------------
class StepEngine:
    def __init__(self):
        self.calls, self.released = [], []

    def step(self, slots, starts, counts, tokens, want):
        self.calls.append((list(slots), list(starts), list(counts), list(tokens), list(want)))
        return np.array([[tokens[w]] for w in want], np.float32).reshape(len(want), 1)

    def release_slot(self, s):
        self.released.append(s)


def test_replay_positions_slots_and_order():
    e = StepEngine()
    r = Replay(e, 2)
    out = r.step([{"id": "a", "tokens": [5, 6, 7], "want": [2, 0]}, {"id": "b", "tokens": [9], "want": []}], [])
    assert out[:, 0].tolist() == [7, 5] and e.calls[-1][1:3] == ([0, 0], [3, 1])
    r.step([{"id": "a", "tokens": [8], "want": [0]}], ["a"])  # b is left out of this step
    assert e.calls[-1][1] == [3] and len(e.released) == 1
    out = r.step([{"id": "c", "tokens": [1, 2], "want": [1]}, {"id": "b", "tokens": [3], "want": [0]}], ["b", "c"])
    assert out[:, 0].tolist() == [2, 3] and e.calls[-1][1] == [0, 1] and sorted(r.free) == [0, 1]
    with pytest.raises(RuntimeError, match="slots"):
        r.step([{"id": i, "tokens": [1], "want": []} for i in "xyz"], [])


# ---- scheduler: mixed steps, limited pool --------------------------------------------------------------
class Tok:
    vocab_size, eos_id, vocab = 1000, -1, {}

    def decode(self, ids):
        return " ".join(str(i) for i in ids)


class MixedEngine:
    """Next token = f(last token, position); records every call; a cache pool of `blocks` blocks."""
    mixed_steps = True
    kv_block_tokens = 4

    def __init__(self, slots, blocks):
        self.log, self.kv_blocks_total = [], blocks
        self.tables = {s: [] for s in range(slots)}
        self.min_free = blocks

    @property
    def kv_blocks_free(self):
        return self.kv_blocks_total - sum(len(t) for t in self.tables.values())

    def block_table(self, s):
        return [100 * s + i for i in range(len(self.tables[s]))] + [-1]

    def release_slot(self, s):
        self.log.append(("release", s))
        self.tables[s] = []

    def _write(self, slot, end):
        while len(self.tables[slot]) * self.kv_block_tokens < end:
            assert self.kv_blocks_free > 0, "pool exhausted"
            self.tables[slot].append(0)
        self.min_free = min(self.min_free, self.kv_blocks_free)

    @staticmethod
    def nxt(tok, pos):
        return (tok * 7 + pos * 3 + 1) % 1000

    def prefill(self, slot, ids, start, want=True):
        self.log.append(("prefill", slot, len(ids), start))
        self._write(slot, start + len(ids))
        l = np.zeros(1000, np.float32)
        l[self.nxt(ids[-1], start + len(ids) - 1)] = 1
        return l

    def decode(self, slots, toks, pos, temps, topk, seed, mask=b"", top_p=None, seeds=None):
        self.log.append(("decode", len(slots)))
        for s, p in zip(slots, pos):
            self._write(s, p + 1)
        return [self.nxt(t, p) for t, p in zip(toks, pos)]

    def step_sample(self, slots, starts, counts, tokens, sample, temps, topk, topp, seeds, mask):
        assert len(set(slots)) == len(slots) and sum(sample) == len(temps) == len(seeds)
        self.log.append(("mixed", list(counts), list(sample)))
        out, at = [], 0
        for s, st, n, k in zip(slots, starts, counts, sample):
            self._write(s, st + n)
            at += n
            if k:
                out.append(self.nxt(tokens[at - 1], st + n - 1))
        return out


def expected(prompt, n):
    out, tok = [], prompt[-1]
    for i in range(n):
        tok = MixedEngine.nxt(tok, len(prompt) - 1 + i)
        out.append(tok)
    return out


def run_all(sched, reqs):
    res, left, ev = {}, [len(reqs)], threading.Event()

    def done(i):
        def f(r):
            res[i] = r
            left[0] -= 1
            if left[0] == 0:
                ev.set()
        return f

    for i, r in enumerate(reqs):
        r.on_done = done(i)
    with sched.cv:
        sched.queue.extend(reqs)
        sched.cv.notify()
    assert ev.wait(20)
    return [res[i] for i in range(len(reqs))]


def test_scheduler_mixes_prompt_chunks_with_decode(monkeypatch):
    monkeypatch.setenv("AIOS_PREFILL_CHUNK", "16")
    eng = MixedEngine(4, 4 * 64)
    sched = Scheduler(eng, Tok(), max_batch=4, max_slots=4, max_ctx=256)
    try:
        prompts = [[i + 3] * n for i, n in enumerate((5, 40, 11, 23))]
        res = run_all(sched, [GenRequest(prompt_ids=p, max_tokens=30) for p in prompts])
    finally:
        sched.close()
    for p, r in zip(prompts, res):
        assert r.token_ids == expected(p, 30) and r.finish_reason == "length"
    mixed = [e for e in eng.log if e[0] == "mixed"]
    assert mixed and all(sum(n for n in e[1] if n > 1) <= 16 for e in mixed)
    assert any(e[1].count(1) >= 1 and max(e[1]) > 1 for e in mixed)         # a portion beside decoded tokens
    assert sum(e[0] == "prefill" for e in eng.log) == 1                     # only the first, with nothing decoding


def test_scheduler_limited_pool_waits_evicts_and_rejects():
    eng = MixedEngine(4, 20)  # 80 tokens for four slots of 64
    sched = Scheduler(eng, Tok(), max_batch=4, max_slots=4, max_ctx=64)
    try:
        prompts = [[i + 3] * 20 for i in range(6)]
        res = run_all(sched, [GenRequest(prompt_ids=p, max_tokens=12) for p in prompts])
        for p, r in zip(prompts, res):
            assert r.token_ids == expected(p, 12), r
        assert any(e[0] == "release" for e in eng.log) and eng.min_free >= 0
        assert not sched.kv_reserved
    finally:
        sched.close()
    eng = MixedEngine(4, 8)
    sched = Scheduler(eng, Tok(), max_batch=4, max_slots=4, max_ctx=64)
    try:
        r = run_all(sched, [GenRequest(prompt_ids=[4] * 20, max_tokens=30)])[0]
        assert r.finish_reason == "error" and "cache pool" in r.error
        r = run_all(sched, [GenRequest(prompt_ids=[4] * 20, max_tokens=5)])[0]
        assert r.token_ids == expected([4] * 20, 5)
    finally:
        sched.close()


def test_cpu_backend_refuses_layered_models(tmp_path):
    from aios_amd.runtime.model_manager import ModelManager

    folder = write_model(tmp_path / "m", MIXED, O.random_weights(MIXED))
    m = asyncio.run(ModelManager(max_batch=2, max_slots=2).load_model("gefazen-cpu", folder + "#cpu"))
    assert m.status == "error" and "GPU only" in m.error
