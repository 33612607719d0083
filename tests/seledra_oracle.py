"""Plain, slow oracle of the Seledra decoder for the tests: one function per mechanism, whole sequences at once, no
cache, no state between calls, no batching, no page, no chunked or fused form, float64 by default.  Shares nothing
with aios_amd: it takes the parsed config.json and a {tensor name: tensor} dict.

Notation: t, s positions; h a head (or, as an argument, a mixer's input); x the residual stream [T, width].
"""
from __future__ import annotations

import math
from typing import Dict, List, Optional

import torch

DT = torch.float64


# ---- mechanisms ----------------------------------------------------------------------------------
def rms(x: torch.Tensor, eps: float) -> torch.Tensor:
    return x / torch.sqrt(x.pow(2).mean(-1, keepdim=True) + eps)


def silu(z: torch.Tensor) -> torch.Tensor:
    return z * torch.sigmoid(z)


def softplus(z: torch.Tensor) -> torch.Tensor:
    return torch.log1p(torch.exp(-z.abs())) + torch.clamp(z, min=0)


def xielu(z: torch.Tensor, p: torch.Tensor, q: torch.Tensor) -> torch.Tensor:
    """z / 2 + softplus(p) z^2 for z > 0, z / 2 + (1/2 + softplus(q)) (e^z - 1 - z) below."""
    neg = torch.clamp(z, max=0)
    return z / 2 + torch.where(z > 0, softplus(p) * z * z, (0.5 + softplus(q)) * (torch.expm1(neg) - neg))


def affine(h: torch.Tensor, w: Dict[str, torch.Tensor], name: str) -> torch.Tensor:
    return h @ w[name].T + w[name + ".b"]


def whole_norm(y: torch.Tensor, g: torch.Tensor, eps: float) -> torch.Tensor:
    """Every row of a projection as one vector, before it becomes heads."""
    return rms(y, eps) * g


def value_norm(v: torch.Tensor, eps: float) -> torch.Tensor:
    return rms(v, eps)


def mix_values(v: torch.Tensor, first: torch.Tensor, lam: torch.Tensor) -> torch.Tensor:
    return (1 - lam) * v + lam * first


def scores(q: torch.Tensor, k: torch.Tensor, scale: float, temp: torch.Tensor) -> torch.Tensor:
    return (k @ q) * scale * temp


def weights(s: torch.Tensor) -> torch.Tensor:
    """Softmax whose denominator has one more term, e^0."""
    return torch.softmax(torch.cat([s, torch.zeros(1, dtype=s.dtype)]), 0)[:-1]


def attention(h: torch.Tensor, w: Dict[str, torch.Tensor], p: str, m: dict, eps: float, shared: dict) -> torch.Tensor:
    """shared: what the layers of one forward pass leave each other ("values": those of the first layer that mixes)."""
    T, H, G, dk, dv = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = whole_norm(affine(h, w, p + "q"), w[p + "q.norm"], eps).view(T, H, dk)
    k = whole_norm(affine(h, w, p + "k"), w[p + "k.norm"], eps).view(T, G, dk)
    v = value_norm(affine(h, w, p + "v").view(T, G, dv), eps)
    if m.get("v_mix"):
        if "values" in shared:
            v = mix_values(v, shared["values"], w[p + "vmix"])
        else:
            shared["values"] = v
    out = torch.zeros(T, H, dv, dtype=h.dtype)
    for n in range(H):
        g = n // (H // G)
        for i in range(T):
            out[i, n] = weights(scores(q[i, n], k[:i + 1, g], m["scale"], w[p + "temp"][n])) @ v[:i + 1, g]
    out = out * torch.sigmoid(h @ w[p + "g"].T)[..., None]
    return out.reshape(T, H * dv) @ w[p + "o"].T


def causal_conv(u: torch.Tensor, k: torch.Tensor) -> torch.Tensor:
    """y_t[c] = sum_j k[c, j] u_{t - (taps - 1) + j}[c], zeros before the first row."""
    T, taps = u.shape[0], k.shape[1]
    pad = torch.cat([torch.zeros(taps - 1, u.shape[1], dtype=u.dtype), u])
    return sum(k[:, j] * pad[j:j + T] for j in range(taps))


def unit(x: torch.Tensor) -> torch.Tensor:
    return x / torch.sqrt(x.pow(2).sum(-1, keepdim=True) + 1e-6)


def decay(z: torch.Tensor, a_log: torch.Tensor, dt_bias: torch.Tensor) -> torch.Tensor:
    return torch.exp(-torch.exp(a_log) * softplus(z + dt_bias))


def delta_rule(g: torch.Tensor, beta: torch.Tensor, k: torch.Tensor, v: torch.Tensor, q: torch.Tensor) -> torch.Tensor:
    """Per head S <- g S, then S += k (beta (v - S^T k))^T, o = S^T q.  g, beta [T, H]; k, q [T, H, n]; v [T, H, m]."""
    S = torch.zeros(k.shape[1], k.shape[2], v.shape[2], dtype=v.dtype)
    out = []
    for t in range(v.shape[0]):
        S = g[t][:, None, None] * S
        u = beta[t][:, None] * (v[t] - (S * k[t][:, :, None]).sum(1))
        S = S + k[t][:, :, None] * u[:, None, :]
        out.append((S * q[t][:, :, None]).sum(1))
    return torch.stack(out)


def delta(h: torch.Tensor, w: Dict[str, torch.Tensor], p: str, m: dict, eps: float, shared: dict) -> torch.Tensor:
    T, H, G, dk, dv = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k, v = (silu(causal_conv(h @ w[p + n].T, w[p + n + ".conv"])) for n in "qkv")
    q = unit(q.view(T, G, dk)) / math.sqrt(dk)
    k = unit(k.view(T, G, dk))
    q, k = (x.repeat_interleave(H // G, 1) for x in (q, k))
    beta = torch.sigmoid(h @ w[p + "b"].T)
    g = decay(h @ w[p + "a"].T, w[p + "A_log"], w[p + "dt_bias"])
    o = rms(delta_rule(g, beta, k, v.view(T, H, dv), q), eps) * w[p + "norm"]
    return (o.reshape(T, H * dv) * silu(h @ w[p + "g"].T)) @ w[p + "o"].T


MIXERS = {"attention": attention, "delta": delta}


def feed_forward(h: torch.Tensor, w: Dict[str, torch.Tensor], p: str) -> torch.Tensor:
    return xielu(h @ w[p + "up"].T, *w[p + "act"]) @ w[p + "down"].T


def embed(w: Dict[str, torch.Tensor], tokens: List[int]) -> torch.Tensor:
    return w["embed"][torch.tensor(tokens)] + w["pos"][:len(tokens)]


def forward(cfg: dict, w: Dict[str, torch.Tensor], tokens: List[int], trace: Optional[list] = None,
            dtype=DT) -> torch.Tensor:
    """Logits [T, vocab]; `trace` collects the residual stream after every layer."""
    w = {k: v.to(dtype) for k, v in w.items()}
    eps, m, shared = cfg["norm"]["eps"], cfg["residual_mult"], {}
    x = embed(w, tokens)
    for i, layer in enumerate(cfg["layers"]):
        p = f"l{i}."
        x = x + m * MIXERS[layer["type"]](rms(x, eps) * w[p + "norm1"], w, p + "mix.", layer["mixer"], eps, shared)
        if layer.get("mlp") is not None:
            x = x + m * feed_forward(rms(x, eps) * w[p + "norm2"], w, p + "mlp.")
        if trace is not None:
            trace.append(x)
    return (rms(x, eps) * w["final.norm"]) @ w["head"].T


def greedy(cfg: dict, w: Dict[str, torch.Tensor], prompt: List[int], n: int) -> List[int]:
    ids = list(prompt)
    for _ in range(n):
        ids.append(int(forward(cfg, w, ids)[-1].argmax()))
    return ids[len(prompt):]


# ---- random models of any size ------------------------------------------------------------------
def make_config(width=96, vocab=211, eps=3e-5, residual_mult=0.8, max_positions=300, layers=None) -> dict:
    return {"architecture": "Seledra", "width": width, "vocab": vocab, "norm": {"eps": eps}, "layers": layers,
            "residual_mult": residual_mult, "max_positions": max_positions}


def dense(ff: int) -> dict:
    return {"kind": "dense", "ff": ff}


def attn_layer(mlp, heads=6, kv_heads=3, dim=20, vdim=28, scale=0.3, v_mix=True) -> dict:
    return {"type": "attention", "mlp": mlp, "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim,
                                                       "scale": scale, "v_mix": v_mix}}


def delta_layer(mlp, heads=6, kv_heads=2, dim=24, vdim=20, conv=4) -> dict:
    return {"type": "delta", "mlp": mlp, "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim,
                                                   "conv": conv}}


def tensor_shapes(cfg: dict) -> Dict[str, tuple]:
    d, V = cfg["width"], cfg["vocab"]
    out = {"embed": (V, d), "pos": (cfg["max_positions"], d), "final.norm": (d,), "head": (V, d)}
    for i, layer in enumerate(cfg["layers"]):
        m, p, mlp = layer["mixer"], f"l{i}.", layer.get("mlp")
        H, G, q = m["heads"], m["kv_heads"], p + "mix."
        out.update({p + "norm1": (d,), q + "o": (d, H * m["vdim"])})
        if layer["type"] == "attention":
            for n, rows in (("q", H * m["dim"]), ("k", G * m["dim"]), ("v", G * m["vdim"])):
                out.update({q + n: (rows, d), q + n + ".b": (rows,)})
            out.update({q + "q.norm": (H * m["dim"],), q + "k.norm": (G * m["dim"],), q + "temp": (H,), q + "g": (H, d)})
            if m.get("v_mix"):
                out[q + "vmix"] = ()
        else:
            for n, rows in (("q", G * m["dim"]), ("k", G * m["dim"]), ("v", H * m["vdim"])):
                out.update({q + n: (rows, d), q + n + ".conv": (rows, m["conv"])})
            out.update({q + "b": (H, d), q + "a": (H, d), q + "A_log": (H,), q + "dt_bias": (H,), q + "norm": (m["vdim"],),
                        q + "g": (H * m["vdim"], d)})
        if mlp is not None:
            out.update({p + "norm2": (d,), p + "mlp.up": (mlp["ff"], d), p + "mlp.down": (d, mlp["ff"]), p + "mlp.act": (2,)})
    return out


def random_weights(cfg: dict, seed: int = 0, qk_gain: float = 1.0) -> Dict[str, torch.Tensor]:
    """bf16 weights; qk_gain > 1 sharpens the attention (single keys stand out)."""
    g = torch.Generator().manual_seed(seed)
    out = {}
    for name, shape in tensor_shapes(cfg).items():
        t = torch.randn(shape, generator=g, dtype=torch.float32)
        last = name.split(".")[-1]
        if last.startswith("norm"):
            t = 1.0 + 0.3 * t
            if name.endswith("q.norm"):
                t = t * qk_gain
        elif name == "embed":
            pass
        elif name == "pos":
            t = 0.5 * t
        elif last == "vmix":
            t = 0.5 + 0.1 * t
        elif last == "temp":
            t = 1.0 + 0.3 * t
        elif last == "act":
            t = 0.5 * t + torch.tensor([0.4, -0.3])
        elif last == "A_log":
            t = t - 1.0
        elif last == "dt_bias":
            t = t - 1.5
        elif last == "conv":
            t = t / math.sqrt(shape[1])
        elif name.endswith((".q.b", ".k.b", ".v.b")):
            t = 0.4 * t
        else:
            t = t / math.sqrt(shape[1])
        out[name] = t.to(torch.bfloat16)
    return out
