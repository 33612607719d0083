"""Movalorn: a small decoder-only language model -- configuration and tensor names.

Token plus token-pair embedding; layers of latent attention (part of the query and key rotated, a sliding window,
a gate per head) or a minGRU recurrence, each followed by a dense MLP (GELU, tanh form), a mixture of
experts with a shared one (SiLU), or nothing; one-number norms before and after every sublayer, whose
result is gated; a span of layers run several times, each pass entered by a projection of the residual
and the embedding.  Every size and constant comes from config.json:

    {"architecture": "Movalorn", "vocab", "width", "norm": {"eps"}, "logit_scale",
     "embedding": {"scale", "bigram": {"buckets", "mul_prev", "mul_cur"}},
     "loop": {"start", "stop", "times"},
     "layers": [{"type": "latent_attention",
                 "mixer": {"heads", "dim", "rot_dim", "vdim", "kv_rank", "scale", "mask": {"size"}, "rot": {"base", "dims"}},
                 or "type": "mingru", "mixer": {"width"},
                 "mlp": {"kind": "dense", "ff"}
                        | {"kind": "moe", "expert": {"ff"}, "router": {"experts", "top", "scale"}, "shared": {"ff"}}
                        | null}, ...]}
"""
from __future__ import annotations

from typing import Dict

from .config import LayerConfig, ModelConfig
from .registry import Architecture

# the design has no table of positions and names no longest sequence: what an engine holds by default
DEFAULT_CTX = 8192

# checkpoint suffix -> engine suffix, per layer
_MIXER = {
    "latent_attention": {"q": "attn_q.weight", "dkv": "attn_kv_a.weight", "dkv.norm": "attn_kv_a_norm.weight",
                         "uk": "attn_k_b.weight", "uv": "attn_v_b.weight", "g": "attn_gate.weight",
                         "o": "attn_output.weight"},
    "mingru": {"z": "rnn_z.weight", "z.b": "rnn_z.bias", "x": "rnn_x.weight", "x.b": "rnn_x.bias",
               "g": "rnn_gate.weight", "o": "rnn_output.weight"},
}
_CLOSING = {"norm{n}": "{s}_norm.weight", "norm{n}b": "{s}_post_norm.weight", "rg{n}": "{s}_resid_gate.weight",
            "rg{n}.b": "{s}_resid_gate.bias"}
_GLU = ("gate", "up", "down")


def _mlp(i: int, mlp) -> dict:
    if mlp is None:
        return dict(ff=0)
    if mlp.get("kind") == "dense":
        return dict(ff=int(mlp["ff"]), act="gelu_tanh")
    if mlp.get("kind") != "moe":
        raise ValueError(f"layer {i}: unknown feed-forward kind {mlp.get('kind')!r}")
    r, shared = mlp["router"], mlp.get("shared")
    return dict(ff=int(mlp["expert"]["ff"]), act="silu", experts=int(r["experts"]), top=int(r["top"]),
                router_scale=float(r["scale"]), correction=True, shared_ff=int(shared["ff"]) if shared else 0)


def _layer(i: int, entry: dict) -> LayerConfig:
    m = entry["mixer"]
    common = dict(parallel=False, norm_scalar=True, post_norm=True, resid_gate=True, sink=False, **_mlp(i, entry.get("mlp")))
    if entry.get("type") == "mingru":
        return LayerConfig(mixer="mingru", width=int(m["width"]), **common)
    if entry.get("type") != "latent_attention":
        raise ValueError(f"layer {i}: unknown mixer type {entry.get('type')!r}")
    window = int(m["mask"]["size"])
    if window < 1:
        raise ValueError(f"layer {i}: a window of {window} tokens")
    return LayerConfig(mixer="latent", heads=int(m["heads"]), dim=int(m["dim"]), vdim=int(m["vdim"]),
                       kv_rank=int(m["kv_rank"]), rot_dim=int(m["rot_dim"]), rot_dims=int(m["rot"]["dims"]),
                       rot_base=float(m["rot"]["base"]), window=window, scale=float(m["scale"]), out_gate="head", **common)


def parse(raw: dict, name: str, shapes=None) -> ModelConfig:
    layers = tuple(_layer(i, e) for i, e in enumerate(raw["layers"]))
    emb, loop = raw["embedding"], raw.get("loop")
    b = emb["bigram"]
    if loop is not None:
        loop = (int(loop["start"]), int(loop["stop"]), int(loop["times"]))
        if not (0 <= loop[0] < loop[1] <= len(layers) and loop[2] >= 1):
            raise ValueError(f"loop {loop} does not fit {len(layers)} layers")
    return ModelConfig(name=name, arch="movalorn", vocab_size=int(raw["vocab"]), d_model=int(raw["width"]),
                       n_layers=len(layers), n_heads=max(l.heads for l in layers), n_kv_heads=1,
                       head_dim=max(l.dim + l.rot_dim for l in layers), d_ff=max(l.ff for l in layers),
                       norm_eps=float(raw["norm"]["eps"]), max_ctx=DEFAULT_CTX, layers=layers, learned_pos=False,
                       embed_scale=float(emb["scale"]), logit_scale=float(raw["logit_scale"]),
                       bigram=(int(b["buckets"]), int(b["mul_prev"]), int(b["mul_cur"])), loop=loop,
                       # the design has no special tokens: nothing is prepended, nothing ends a generation
                       bos_id=-1, eos_id=-1)


def tensor_names(raw: dict) -> Dict[str, str]:
    out = {"embed": "token_embd.weight", "bigram": "bigram_embd.weight", "final.norm": "output_norm.weight",
           "head": "output.weight"}
    if raw.get("loop") is not None:
        out.update({"loop.in": "loop_in.weight", "loop.step": "loop_step.weight"})
    for i, e in enumerate(raw["layers"]):
        names = {f"mix.{k}": v for k, v in _MIXER[e["type"]].items()}
        mlp = e.get("mlp")
        for n, s in ((1, "attn"), (2, "ffn")):
            if n == 1 or mlp is not None:
                names.update({k.format(n=n): v.format(s=s) for k, v in _CLOSING.items()})
        if mlp is not None and mlp["kind"] == "dense":
            names.update({f"mlp.{k}": f"ffn_{k}.weight" for k in _GLU})
        elif mlp is not None:
            names.update({"mlp.router": "ffn_gate_inp.weight", "mlp.correction": "exp_probs_b.bias"})
            if mlp.get("shared"):
                names.update({f"mlp.shared.{k}": f"ffn_{k}_shexp.weight" for k in _GLU})
            for x in range(int(mlp["router"]["experts"])):
                names.update({f"mlp.e{x}.{k}": f"ffn_{k}.{x}.weight" for k in _GLU})
        out.update({f"l{i}.{k}": f"blk.{i}.{v}" for k, v in names.items()})
    return out


ARCHITECTURE = Architecture(parse=parse, tensor_names=tensor_names)
