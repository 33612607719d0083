"""Plain, slow oracle of the Gefazen decoder for the tests: one function per mechanism, whole
sequences at once, no cache, no batching, no page, no fused or absorbed form, float64 by default.
Shares nothing with aios_amd: it takes the parsed config.json and a {tensor name: tensor} dict.

Notation: t, s positions; h a head; r the latent width; x the residual stream [T, width].
"""
from __future__ import annotations

import math
from typing import Dict, List, Optional

import torch

DT = torch.float64


def rms_norm(x: torch.Tensor, w: torch.Tensor, eps: float) -> torch.Tensor:
    return x / torch.sqrt(x.pow(2).mean(-1, keepdim=True) + eps) * w


def gelu_tanh(z: torch.Tensor) -> torch.Tensor:
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def embed(tokens: List[int], table: torch.Tensor, pos_table: torch.Tensor) -> torch.Tensor:
    return torch.stack([table[t] + pos_table[p] for p, t in enumerate(tokens)])


def sink_softmax(scores: torch.Tensor, sink: float) -> torch.Tensor:
    """Weights of the visible keys: exp(a_s) / (exp(sink) + sum exp(a)); they sum to less than 1."""
    top = max(float(scores.max()), float(sink))
    e = torch.exp(scores - top)
    return e / (e.sum() + math.exp(float(sink) - top))


def latent(h: torch.Tensor, w: Dict[str, torch.Tensor], p: str, eps: float) -> torch.Tensor:
    """What a token leaves behind for later ones: its normalised down-projection."""
    return rms_norm(h @ w[p + "dkv"].T, w[p + "dkv.norm"], eps)


def latent_attention(h: torch.Tensor, w: Dict[str, torch.Tensor], p: str, mx: dict, eps: float) -> torch.Tensor:
    T, H, dk, dv = h.shape[0], mx["heads"], mx["dim"], mx["vdim"]
    q = (h @ w[p + "q"].T).view(T, H, dk)
    c = latent(h, w, p, eps)
    k = (c @ w[p + "uk"].T).view(T, H, dk)
    v = (c @ w[p + "uv"].T).view(T, H, dv)
    out = torch.zeros(T, H, dv, dtype=h.dtype)
    for i in range(T):
        for n in range(H):
            a = (k[: i + 1, n] @ q[i, n]) * mx["scale"]
            out[i, n] = sink_softmax(a, float(w[p + "sink"][n])) @ v[: i + 1, n]
    gate = torch.sigmoid(h @ w[p + "g"].T)
    return (out.reshape(T, H * dv) * gate) @ w[p + "o"].T


def gated_mlp(h: torch.Tensor, w: Dict[str, torch.Tensor], p: str) -> torch.Tensor:
    return (gelu_tanh(h @ w[p + "gate"].T) * (h @ w[p + "up"].T)) @ w[p + "down"].T


def owner(layers: List[dict], i: int) -> int:
    """The layer whose tensors layer i uses."""
    while "weights_of" in layers[i]:
        i = layers[i]["weights_of"]
    return i


def forward(cfg: dict, w: Dict[str, torch.Tensor], tokens: List[int], trace: Optional[list] = None) -> torch.Tensor:
    """Logits [T, vocab]; `trace` collects the residual stream after every layer."""
    w = {k: v.to(DT) for k, v in w.items()}
    eps = cfg["norm"]["eps"]
    x = embed(tokens, w["embed"], w["pos"])
    for i, layer in enumerate(cfg["layers"]):
        p = f"l{owner(cfg['layers'], i)}."
        h = rms_norm(x, w[p + "norm1"], eps)
        y = latent_attention(h, w, p + "mix.", layer["mixer"], eps)
        if layer.get("mlp") is not None:
            y = y + gated_mlp(h, w, p + "mlp.")
        x = x + y
        if trace is not None:
            trace.append(x)
    return rms_norm(x, w["final.norm"], eps) @ w["head"].T


def greedy(cfg: dict, w: Dict[str, torch.Tensor], prompt: List[int], n: int) -> List[int]:
    ids = list(prompt)
    for _ in range(n):
        ids.append(int(forward(cfg, w, ids)[-1].argmax()))
    return ids[len(prompt):]


# ---- random models of any size ------------------------------------------------------------------
def make_config(width=96, vocab=211, max_positions=512, eps=3e-5, layers=None) -> dict:
    return {"architecture": "Gefazen", "width": width, "vocab": vocab, "max_positions": max_positions,
            "norm": {"eps": eps}, "layers": layers}


def make_layer(heads=3, dim=24, vdim=40, kv_rank=56, scale=0.17, ff: Optional[int] = 72,
               weights_of: Optional[int] = None) -> dict:
    d = {"type": "latent_attention",
         "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "kv_rank": kv_rank, "scale": scale},
         "mlp": None if ff is None else {"kind": "dense", "ff": ff}}
    if weights_of is not None:
        d["weights_of"] = weights_of
    return d


def tensor_shapes(cfg: dict) -> Dict[str, tuple]:
    d, V = cfg["width"], cfg["vocab"]
    out = {"embed": (V, d), "pos": (cfg["max_positions"], d), "final.norm": (d,), "head": (V, d)}
    for i, layer in enumerate(cfg["layers"]):
        if "weights_of" in layer:
            continue
        m, p = layer["mixer"], f"l{i}."
        H, dk, dv, r = m["heads"], m["dim"], m["vdim"], m["kv_rank"]
        out.update({p + "norm1": (d,), p + "mix.q": (H * dk, d), p + "mix.dkv": (r, d), p + "mix.dkv.norm": (r,),
                    p + "mix.uk": (H * dk, r), p + "mix.uv": (H * dv, r), p + "mix.sink": (H,),
                    p + "mix.g": (H * dv, d), p + "mix.o": (d, H * dv)})
        if layer.get("mlp") is not None:
            f = layer["mlp"]["ff"]
            out.update({p + "mlp.gate": (f, d), p + "mlp.up": (f, d), p + "mlp.down": (d, f)})
    return out


def random_weights(cfg: dict, seed: int = 0, qk_gain: float = 1.0) -> Dict[str, torch.Tensor]:
    """bf16 weights; qk_gain > 1 sharpens the attention (single keys stand out)."""
    g = torch.Generator().manual_seed(seed)
    out = {}
    for name, shape in tensor_shapes(cfg).items():
        t = torch.randn(*shape, generator=g, dtype=torch.float32)
        if name.endswith(("norm1", ".norm")):
            t = 1.0 + 0.2 * t
        elif name in ("embed", "pos"):
            t = t * (1.0 if name == "embed" else 0.5)
        elif name.endswith(".sink"):
            t = t * 1.5
        else:
            t = t / math.sqrt(shape[1])
            if name.endswith((".q", ".uk")):
                t = t * qk_gain
        out[name] = t.to(torch.bfloat16)
    return out
