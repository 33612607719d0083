"""Sinisun: a small decoder-only language model -- configuration and tensor names.

Layers of Mamba-2 (state-space duality), or of grouped-query attention (half-rotated positions, soft-capped scores within
chunks of positions, a sink and a gate per head) beside gated linear attention, whose results are added with two scales;
each followed by an MLP without a gate (square of relu, biases), or nothing.  A span of layers may run several times; every
pass but the first is entered by adding the embedding to the residual.  Sizes and constants come from config.json, the
width of the linear attention's decay projection from its tensor:

    {"architecture": "Sinisun", "vocab", "width", "norm": {"eps"}, "loop": {"start", "stop", "times"} | null,
     "layers": [{"type": "mamba2", "mixer": {"heads", "vdim", "state", "groups", "norm_groups", "conv"}}
                or {"type": "parallel",
                    "mixer": {"left": {"heads", "kv_heads", "dim", "vdim", "rot": {"base", "dims"}, "mask": {"size"},
                                       "scale", "softcap"},
                              "right": {"heads", "dim", "vdim", "tau"}, "left_scale", "right_scale"}},
                with "mlp": {"kind": "dense", "ff"} | null, ...]}
"""
from __future__ import annotations

from typing import Dict

from .config import LayerConfig, LinConfig, ModelConfig
from .registry import Architecture

# the design has no table of positions and names no longest sequence: what an engine holds by default
DEFAULT_CTX = 8192

# checkpoint suffix -> engine suffix, per layer
_MIXER = {
    "mamba2": {"in": "ssm_in.weight", "conv": "ssm_conv1d.weight", "conv.b": "ssm_conv1d.bias", "dt_bias": "ssm_dt.bias",
               "A_log": "ssm_a_log.bias", "D": "ssm_d.bias", "norm": "ssm_norm.weight", "o": "ssm_out.weight"},
    "parallel": {**{f"left.{k}{b}": f"attn_{n}{s}" for k, n in (("q", "q"), ("k", "k"), ("v", "v"), ("o", "output"))
                    for b, s in (("", ".weight"), (".b", ".bias"))},
                 "left.sink": "attn_sinks.weight", "left.g": "attn_gate.weight",
                 **{f"right.{k}": f"gla_{n}.weight" for k, n in (("q", "q"), ("k", "k"), ("v", "v"), ("g", "gate"),
                                                                 ("a1", "a1"), ("a2", "a2"), ("norm", "norm"),
                                                                 ("o", "output"))},
                 "right.a2.b": "gla_a2.bias"},
}
_MLP = {"up": "ffn_up.weight", "up.b": "ffn_up.bias", "down": "ffn_down.weight", "down.b": "ffn_down.bias"}


def _mlp(i: int, mlp) -> dict:
    if mlp is None:
        return dict(ff=0)
    if mlp.get("kind") != "dense":
        raise ValueError(f"layer {i}: unknown feed-forward kind {mlp.get('kind')!r}")
    return dict(ff=int(mlp["ff"]))


def _layer(i: int, entry: dict, shapes) -> LayerConfig:
    m = entry["mixer"]
    common = dict(parallel=False, gated=False, act="relu2", mlp_bias=True, **_mlp(i, entry.get("mlp")))
    if entry.get("type") == "mamba2":
        lin = LinConfig(heads=int(m["heads"]), groups=int(m["groups"]), dim=int(m["state"]), vdim=int(m["vdim"]),
                        conv=int(m["conv"]), norm_groups=int(m["norm_groups"]))
        if lin.heads % lin.groups or (lin.heads * lin.vdim) % lin.norm_groups:
            raise ValueError(f"layer {i}: heads in {lin.groups} groups, norm in {lin.norm_groups} parts")
        return LayerConfig(mixer="mamba2", lin=lin, sink=False, out_gate="none", **common)
    if entry.get("type") != "parallel":
        raise ValueError(f"layer {i}: unknown mixer type {entry.get('type')!r}")
    l, r = m["left"], m["right"]
    chunk = int(l["mask"]["size"])
    if chunk < 1:
        raise ValueError(f"layer {i}: chunks of {chunk} tokens")
    if int(l["heads"]) % int(l["kv_heads"]):
        raise ValueError(f"layer {i}: {l['heads']} query heads for {l['kv_heads']} key heads")
    lin = LinConfig(heads=int(r["heads"]), groups=int(r["heads"]), dim=int(r["dim"]), vdim=int(r["vdim"]), tau=float(r["tau"]),
                    rank=int(shapes[f"l{i}.mix.right.a1"][0]))
    return LayerConfig(mixer="gqa", beside="gla", mixer_scale=float(m["left_scale"]), beside_scale=float(m["right_scale"]),
                       lin=lin, heads=int(l["heads"]), kv_heads=int(l["kv_heads"]), dim=int(l["dim"]), vdim=int(l["vdim"]),
                       rot_dims=int(l["rot"]["dims"]), rot_base=float(l["rot"]["base"]), chunk=chunk, scale=float(l["scale"]),
                       softcap=float(l["softcap"]), attn_bias=True, sink=True, out_gate="head", **common)


def parse(raw: dict, name: str, shapes) -> ModelConfig:
    layers = tuple(_layer(i, e, shapes) for i, e in enumerate(raw["layers"]))
    loop = raw.get("loop")
    if loop is not None:
        loop = (int(loop["start"]), int(loop["stop"]), int(loop["times"]))
        if not (0 <= loop[0] < loop[1] <= len(layers) and loop[2] >= 1):
            raise ValueError(f"loop {loop} does not fit {len(layers)} layers")
    return ModelConfig(name=name, arch="sinisun", vocab_size=int(raw["vocab"]), d_model=int(raw["width"]),
                       n_layers=len(layers), n_heads=max(l.heads for l in layers), n_kv_heads=max(l.kv_heads for l in layers),
                       head_dim=max(l.dim for l in layers), d_ff=max(l.ff for l in layers),
                       norm_eps=float(raw["norm"]["eps"]), max_ctx=DEFAULT_CTX, layers=layers, learned_pos=False, loop=loop,
                       loop_add=True,
                       # the design has no special tokens: nothing is prepended, nothing ends a generation
                       bos_id=-1, eos_id=-1)


def tensor_names(raw: dict) -> Dict[str, str]:
    out = {"embed": "token_embd.weight", "final.norm": "output_norm.weight", "head": "output.weight"}
    for i, e in enumerate(raw["layers"]):
        names = {"norm1": "attn_norm.weight", **{f"mix.{k}": v for k, v in _MIXER[e["type"]].items()}}
        if e.get("mlp") is not None:
            names.update({"norm2": "ffn_norm.weight", **{f"mlp.{k}": v for k, v in _MLP.items()}})
        out.update({f"l{i}.{k}": f"blk.{i}.{v}" for k, v in names.items()})
    return out


ARCHITECTURE = Architecture(parse=parse, tensor_names=tensor_names)
