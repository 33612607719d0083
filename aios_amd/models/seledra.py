"""Seledra: a small decoder-only language model -- configuration and tensor names.

Layers of grouped-query attention without rotation (queries and keys normalised over the whole projection, values per head,
scores times a number per head, one added to the softmax's denominator, values mixed with the first such layer's, a gate per
head), or of the gated delta rule (short convolutions, unit queries and keys, a decay and a strength per head); each followed by
an MLP without a gate (xIELU), or nothing.  Every sublayer's result is multiplied by one constant before it is added; learned
positions.  Sizes and constants come from config.json:

    {"architecture": "Seledra", "vocab", "width", "norm": {"eps"}, "residual_mult", "max_positions",
     "layers": [{"type": "attention", "mixer": {"heads", "kv_heads", "dim", "vdim", "scale", "v_mix"}}
                or {"type": "delta", "mixer": {"heads", "kv_heads", "dim", "vdim", "conv"}}
                with "mlp": {"kind": "dense", "ff"} | null, ...]}
"""
from __future__ import annotations

from typing import Dict

from .config import LayerConfig, LinConfig, ModelConfig
from .registry import Architecture

# checkpoint suffix -> engine suffix, per layer ("mix.vmix" only where values are mixed)
_MIXER = {
    "attention": {**{f"{k}{b}": f"attn_{k}{s}" for k in "qkv" for b, s in (("", ".weight"), (".b", ".bias"))},
                  "q.norm": "attn_q_norm.weight", "k.norm": "attn_k_norm.weight", "temp": "attn_temp.weight",
                  "vmix": "attn_v_mix.weight", "g": "attn_gate.weight", "o": "attn_output.weight"},
    "delta": {**{f"{k}{b}": f"delta_{k}{s}" for k in "qkv" for b, s in (("", ".weight"), (".conv", "_conv1d.weight"))},
              "b": "delta_b.weight", "a": "delta_a.weight", "A_log": "delta_a_log.bias", "dt_bias": "delta_dt.bias",
              "norm": "delta_norm.weight", "g": "delta_gate.weight", "o": "delta_output.weight"},
}
_MLP = {"up": "ffn_up.weight", "down": "ffn_down.weight", "act": "ffn_act.bias"}


def _mlp(i: int, mlp) -> dict:
    if mlp is None:
        return dict(ff=0)
    if mlp.get("kind") != "dense":
        raise ValueError(f"layer {i}: unknown feed-forward kind {mlp.get('kind')!r}")
    return dict(ff=int(mlp["ff"]))


def _layer(i: int, entry: dict, mult: float) -> LayerConfig:
    m, kind = entry["mixer"], entry.get("type")
    if kind not in _MIXER:
        raise ValueError(f"layer {i}: unknown mixer type {kind!r}")
    heads, kv = int(m["heads"]), int(m["kv_heads"])
    if heads % kv:
        raise ValueError(f"layer {i}: {heads} heads for {kv} key heads")
    common = dict(parallel=False, gated=False, act="xielu", mixer_scale=mult, mlp_scale=mult, sink=False, **_mlp(i, entry.get("mlp")))
    if kind == "delta":
        lin = LinConfig(heads=heads, groups=kv, dim=int(m["dim"]), vdim=int(m["vdim"]), conv=int(m["conv"]))
        return LayerConfig(mixer="delta", lin=lin, out_gate="none", **common)
    return LayerConfig(mixer="gqa", heads=heads, kv_heads=kv, dim=int(m["dim"]), vdim=int(m["vdim"]), scale=float(m["scale"]),
                       sink_one=True, out_gate="head", attn_bias=True, out_bias=False, qk_norm=True, v_norm=True, head_temp=True,
                       v_mix=bool(m.get("v_mix", False)), **common)


def parse(raw: dict, name: str, shapes=None) -> ModelConfig:
    layers = tuple(_layer(i, e, float(raw["residual_mult"])) for i, e in enumerate(raw["layers"]))
    mixed = [l for l in layers if l.v_mix]
    if any((l.kv_heads, l.vdim) != (mixed[0].kv_heads, mixed[0].vdim) for l in mixed):
        raise ValueError("layers whose values are mixed differ in value heads")
    return ModelConfig(name=name, arch="seledra", vocab_size=int(raw["vocab"]), d_model=int(raw["width"]), n_layers=len(layers),
                       n_heads=max(l.heads for l in layers), n_kv_heads=max(l.kv_heads for l in layers),
                       head_dim=max(l.dim for l in layers), d_ff=max(l.ff for l in layers),
                       norm_eps=float(raw["norm"]["eps"]), max_ctx=int(raw["max_positions"]), layers=layers, learned_pos=True,
                       # the design has no special tokens: nothing is prepended, nothing ends a generation
                       bos_id=-1, eos_id=-1)


def tensor_names(raw: dict) -> Dict[str, str]:
    out = {"embed": "token_embd.weight", "pos": "position_embd.weight", "final.norm": "output_norm.weight", "head": "output.weight"}
    for i, e in enumerate(raw["layers"]):
        mixer = {k: v for k, v in _MIXER[e["type"]].items() if k != "vmix" or e["mixer"].get("v_mix")}
        names = {"norm1": "attn_norm.weight", **{f"mix.{k}": v for k, v in mixer.items()}}
        if e.get("mlp") is not None:
            names.update({"norm2": "ffn_norm.weight", **{f"mlp.{k}": v for k, v in _MLP.items()}})
        out.update({f"l{i}.{k}": f"blk.{i}.{v}" for k, v in names.items()})
    return out


ARCHITECTURE = Architecture(parse=parse, tensor_names=tensor_names)
