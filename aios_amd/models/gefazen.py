"""Gefazen: a small decoder-only language model -- configuration and tensor names.

Learned positions added to the embedding; parallel layers (mixer and MLP read one RMS norm and are added
together); latent attention without positions, with a softmax sink per head and an output gate; a gated
MLP with GELU (tanh form), or none; a layer may run with another layer's weights.  Every size and
constant comes from config.json:

    {"architecture": "Gefazen", "vocab", "width", "max_positions", "norm": {"eps"},
     "layers": [{"type": "latent_attention",
                 "mixer": {"heads", "dim", "vdim", "kv_rank", "scale"},
                 "mlp": {"kind": "dense", "ff"} | null,
                 "weights_of": j (optional)}, ...]}
"""
from __future__ import annotations

from typing import Dict

from .config import LayerConfig, ModelConfig
from .registry import Architecture

# checkpoint suffix -> engine suffix, per layer
_LAYER = {
    "norm1": "attn_norm.weight",
    "mix.q": "attn_q.weight",
    "mix.dkv": "attn_kv_a.weight",
    "mix.dkv.norm": "attn_kv_a_norm.weight",
    "mix.uk": "attn_k_b.weight",
    "mix.uv": "attn_v_b.weight",
    "mix.sink": "attn_sinks.weight",
    "mix.g": "attn_gate.weight",
    "mix.o": "attn_output.weight",
}
_MLP = {"mlp.gate": "ffn_gate.weight", "mlp.up": "ffn_up.weight", "mlp.down": "ffn_down.weight"}


def _layer(i: int, entry: dict) -> LayerConfig:
    if entry.get("type") != "latent_attention":
        raise ValueError(f"layer {i}: unknown mixer type {entry.get('type')!r}")
    m, mlp = entry["mixer"], entry.get("mlp")
    if mlp is not None and mlp.get("kind") != "dense":
        raise ValueError(f"layer {i}: unknown feed-forward kind {mlp.get('kind')!r}")
    w = entry.get("weights_of")
    return LayerConfig(mixer="latent", heads=int(m["heads"]), dim=int(m["dim"]), vdim=int(m["vdim"]),
                       kv_rank=int(m["kv_rank"]), scale=float(m["scale"]), sink=True, out_gate="element",
                       ff=0 if mlp is None else int(mlp["ff"]), act="gelu_tanh", weights_of=-1 if w is None else int(w))


def parse(raw: dict, name: str, shapes=None) -> ModelConfig:
    layers = tuple(_layer(i, e) for i, e in enumerate(raw["layers"]))
    for i, l in enumerate(layers):
        seen, j = {i}, i
        while layers[j].weights_of >= 0:
            j = layers[j].weights_of
            if j >= len(layers) or j in seen:
                raise ValueError(f"layer {i}: weights_of names no layer with weights")
            seen.add(j)
    return ModelConfig(name=name, arch="gefazen", vocab_size=int(raw["vocab"]), d_model=int(raw["width"]),
                       n_layers=len(layers), n_heads=max(l.heads for l in layers), n_kv_heads=1,
                       head_dim=max(l.dim for l in layers), d_ff=max(l.ff for l in layers),
                       norm_eps=float(raw["norm"]["eps"]), max_ctx=int(raw["max_positions"]), layers=layers,
                       # the design has no special tokens: nothing is prepended, nothing ends a generation
                       bos_id=-1, eos_id=-1)


def tensor_names(raw: dict) -> Dict[str, str]:
    out = {"embed": "token_embd.weight", "pos": "position_embd.weight", "final.norm": "output_norm.weight",
           "head": "output.weight"}
    for i, e in enumerate(raw["layers"]):
        if e.get("weights_of") is not None:
            continue
        names = dict(_LAYER, **(_MLP if e.get("mlp") is not None else {}))
        out.update({f"l{i}.{k}": f"blk.{i}.{v}" for k, v in names.items()})
    return out


ARCHITECTURE = Architecture(parse=parse, tensor_names=tensor_names)
