"""Plain, slow oracle of the Sinisun decoder for the tests: one function per mechanism, whole sequences at once, no
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


def rms_parts(x: torch.Tensor, parts: int, eps: float) -> torch.Tensor:
    """Every one of `parts` equal pieces of a row by its own root mean square."""
    return rms(x.reshape(x.shape[0], parts, -1), eps).reshape(x.shape)


def silu(z: torch.Tensor) -> torch.Tensor:
    return z * torch.sigmoid(z)


def softplus(z: torch.Tensor) -> torch.Tensor:
    return torch.log1p(torch.exp(-z.abs())) + torch.clamp(z, min=0)


def linear(h: torch.Tensor, w: Dict[str, torch.Tensor], name: str) -> torch.Tensor:
    y = h @ w[name].T
    return y + w[name + ".b"] if name + ".b" in w else y


def causal_conv(u: torch.Tensor, k: torch.Tensor, b: torch.Tensor) -> torch.Tensor:
    """y_t[c] = b[c] + sum_j k[c, j] u_{t - (taps - 1) + j}[c], zeros before the first row."""
    T, taps = u.shape[0], k.shape[1]
    pad = torch.cat([torch.zeros(taps - 1, u.shape[1], dtype=u.dtype), u])
    return b + sum(k[:, j] * pad[j:j + T] for j in range(taps))


def decayed_outer(decay: torch.Tensor, k: torch.Tensor, v: torch.Tensor, q: torch.Tensor,
                  s0: Optional[torch.Tensor] = None) -> torch.Tensor:
    """S_t = decay_t S_{t-1} + k_t v_t^T per head, o_t = S_t^T q_t.  decay, k, q [T, H, n]; v [T, H, m]."""
    S = torch.zeros(k.shape[1], k.shape[2], v.shape[2], dtype=v.dtype) if s0 is None else s0
    out = []
    for t in range(v.shape[0]):
        S = decay[t][:, :, None] * S + k[t][:, :, None] * v[t][:, None, :]
        out.append((S * q[t][:, :, None]).sum(1))
    return torch.stack(out)


def mamba2(h: torch.Tensor, w: Dict[str, torch.Tensor], p: str, m: dict, eps: float) -> torch.Tensor:
    T, H, dv, N, G = h.shape[0], m["heads"], m["vdim"], m["state"], m["groups"]
    inner = H * dv
    y = h @ w[p + "in"].T
    z, u, dt = y[:, :inner], y[:, inner:2 * inner + 2 * G * N], y[:, 2 * inner + 2 * G * N:]
    u = silu(causal_conv(u, w[p + "conv"], w[p + "conv.b"]))
    x = u[:, :inner].reshape(T, H, dv)
    B = u[:, inner:inner + G * N].reshape(T, G, N).repeat_interleave(H // G, 1)
    C = u[:, inner + G * N:].reshape(T, G, N).repeat_interleave(H // G, 1)
    dt = softplus(dt + w[p + "dt_bias"])
    decay = torch.exp(-torch.exp(w[p + "A_log"]) * dt)[..., None].expand(T, H, N)
    o = decayed_outer(decay, B * dt[..., None], x, C) + w[p + "D"][:, None] * x
    o = rms_parts(o.reshape(T, inner) * silu(z), m["norm_groups"], eps) * w[p + "norm"]
    return o @ w[p + "o"].T


def rotate_half(v: torch.Tensor, base: float, dims: int) -> torch.Tensor:
    """v [T, H, n] with row t at position t: pairs (i, i + dims / 2), i < dims / 2, turned by t base^(-2i/dims)."""
    out = v.clone()
    for i in range(dims // 2):
        a = (torch.arange(v.shape[0], dtype=v.dtype) * base ** (-2.0 * i / dims))[:, None]
        x, y = v[..., i], v[..., i + dims // 2]
        out[..., i] = x * torch.cos(a) - y * torch.sin(a)
        out[..., i + dims // 2] = y * torch.cos(a) + x * torch.sin(a)
    return out


def visible(i: int, size: int) -> range:
    """Keys of query i: those of its own chunk of `size` positions, up to itself."""
    return range(i // size * size, i + 1)


def soft_cap(score: torch.Tensor, cap: float) -> torch.Tensor:
    return cap * torch.tanh(score / cap)


def sink_weights(score: torch.Tensor, sink: torch.Tensor) -> torch.Tensor:
    """Softmax whose denominator has exp(sink) beside the keys' terms."""
    return torch.softmax(torch.cat([score, sink.reshape(1)]), 0)[:-1]


def attention(h: torch.Tensor, w: Dict[str, torch.Tensor], p: str, m: dict) -> torch.Tensor:
    T, H, G, dk, dv = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = rotate_half(linear(h, w, p + "q").view(T, H, dk), m["rot"]["base"], m["rot"]["dims"])
    k = rotate_half(linear(h, w, p + "k").view(T, G, dk), m["rot"]["base"], m["rot"]["dims"])
    v = linear(h, w, p + "v").view(T, G, dv)
    out = torch.zeros(T, H, dv, dtype=h.dtype)
    for i in range(T):
        see = visible(i, m["mask"]["size"])
        a, b = see.start, see.stop
        for n in range(H):
            g = n // (H // G)
            score = soft_cap((k[a:b, g] @ q[i, n]) * m["scale"], m["softcap"])
            out[i, n] = sink_weights(score, w[p + "sink"][n]) @ v[a:b, g]
    out = out * torch.sigmoid(h @ w[p + "g"].T)[..., None]
    return linear(out.reshape(T, H * dv), w, p + "o")


def gla_decay(h: torch.Tensor, w: Dict[str, torch.Tensor], p: str, m: dict) -> torch.Tensor:
    z = linear(h @ w[p + "a1"].T, w, p + "a2")
    return torch.sigmoid(z).pow(1.0 / m["tau"]).view(h.shape[0], m["heads"], m["dim"])


def gated_linear_attention(h: torch.Tensor, w: Dict[str, torch.Tensor], p: str, m: dict, eps: float) -> torch.Tensor:
    T, H, dk, dv = h.shape[0], m["heads"], m["dim"], m["vdim"]
    q = (h @ w[p + "q"].T).view(T, H, dk) / math.sqrt(dk)
    k, v = (h @ w[p + "k"].T).view(T, H, dk), (h @ w[p + "v"].T).view(T, H, dv)
    o = rms(decayed_outer(gla_decay(h, w, p, m), k, v, q), eps) * w[p + "norm"]
    return (o.reshape(T, H * dv) * silu(h @ w[p + "g"].T)) @ w[p + "o"].T


def parallel(h: torch.Tensor, w: Dict[str, torch.Tensor], p: str, m: dict, eps: float) -> torch.Tensor:
    return (m["left_scale"] * attention(h, w, p + "left.", m["left"]) +
            m["right_scale"] * gated_linear_attention(h, w, p + "right.", m["right"], eps))


MIXERS = {"mamba2": mamba2, "parallel": parallel}


def feed_forward(h: torch.Tensor, w: Dict[str, torch.Tensor], p: str) -> torch.Tensor:
    return linear(torch.relu(linear(h, w, p + "up")) ** 2, w, p + "down")


def schedule(cfg: dict) -> List[tuple]:
    """(layer, pass) in running order; pass -1 outside the loop."""
    n, lp = len(cfg["layers"]), cfg.get("loop")
    if not lp:
        return [(i, -1) for i in range(n)]
    return ([(i, -1) for i in range(lp["start"])] +
            [(i, t) for t in range(lp["times"]) for i in range(lp["start"], lp["stop"])] +
            [(i, -1) for i in range(lp["stop"], n)])


def forward(cfg: dict, w: Dict[str, torch.Tensor], tokens: List[int], trace: Optional[list] = None,
            dtype=DT) -> torch.Tensor:
    """Logits [T, vocab]; `trace` collects the residual stream after every layer run."""
    w = {k: v.to(dtype) for k, v in w.items()}
    eps = cfg["norm"]["eps"]
    x = x0 = w["embed"][torch.tensor(tokens)]
    for i, t in schedule(cfg):
        if t > 0 and i == cfg["loop"]["start"]:
            x = x + x0
        layer, p = cfg["layers"][i], f"l{i}."
        h = rms(x, eps) * w[p + "norm1"]
        x = x + MIXERS[layer["type"]](h, w, p + "mix.", layer["mixer"], eps)
        if layer.get("mlp") is not None:
            x = x + feed_forward(rms(x, eps) * w[p + "norm2"], w, p + "mlp.")
        if trace is not None:
            trace.append(x)
    return (rms(x, eps) * w["final.norm"]) @ w["head"].T


def greedy(cfg: dict, w: Dict[str, torch.Tensor], prompt: List[int], n: int) -> List[int]:
    ids = list(prompt)
    for _ in range(n):
        ids.append(int(forward(cfg, w, ids)[-1].argmax()))
    return ids[len(prompt):]


# ---- random models of any size ------------------------------------------------------------------
def make_config(width=96, vocab=211, eps=3e-5, layers=None, loop=None) -> dict:
    return {"architecture": "Sinisun", "width": width, "vocab": vocab, "norm": {"eps": eps}, "layers": layers,
            "loop": None if loop is None else dict(zip(("start", "stop", "times"), loop))}


def dense(ff: int) -> dict:
    return {"kind": "dense", "ff": ff}


def mamba_layer(mlp, heads=4, vdim=24, state=20, groups=2, norm_groups=4, conv=3) -> dict:
    return {"type": "mamba2", "mlp": mlp, "mixer": {"heads": heads, "vdim": vdim, "state": state, "groups": groups,
                                                    "norm_groups": norm_groups, "conv": conv}}


def attn(heads=6, kv_heads=2, dim=40, vdim=24, rot=28, base=3000.0, size=17, scale=0.21, softcap=9.0) -> dict:
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "rot": {"base": base, "dims": rot},
            "mask": {"size": size}, "scale": scale, "softcap": softcap}


def gla(heads=3, dim=24, vdim=40, tau=5.0, rank=12) -> dict:
    return {"heads": heads, "dim": dim, "vdim": vdim, "tau": tau, "rank": rank}


def parallel_layer(mlp, left=None, right=None, left_scale=0.7, right_scale=1.2) -> dict:
    right = dict(right or gla())
    rank = right.pop("rank")  # (a size that only the tensors' shapes give)
    return {"type": "parallel", "mlp": mlp, "_rank": rank,
            "mixer": {"left": left or attn(), "right": right, "left_scale": left_scale, "right_scale": right_scale}}


def plain(cfg: dict) -> dict:
    """The configuration as config.json has it."""
    return dict(cfg, layers=[{k: v for k, v in l.items() if k != "_rank"} for l in cfg["layers"]])


def tensor_shapes(cfg: dict) -> Dict[str, tuple]:
    d, V = cfg["width"], cfg["vocab"]
    out = {"embed": (V, d), "final.norm": (d,), "head": (V, d)}

    def biased(name, n, k):
        out.update({name: (n, k), name + ".b": (n,)})

    for i, layer in enumerate(cfg["layers"]):
        m, p, mlp = layer["mixer"], f"l{i}.", layer.get("mlp")
        out[p + "norm1"] = (d,)
        if layer["type"] == "mamba2":
            H, inner, gn = m["heads"], m["heads"] * m["vdim"], m["groups"] * m["state"]
            out.update({p + "mix.in": (2 * inner + 2 * gn + H, d), p + "mix.conv": (inner + 2 * gn, m["conv"]),
                        p + "mix.conv.b": (inner + 2 * gn,), p + "mix.dt_bias": (H,), p + "mix.A_log": (H,),
                        p + "mix.D": (H,), p + "mix.norm": (inner,), p + "mix.o": (d, inner)})
        else:
            l, r, q = m["left"], m["right"], p + "mix.left."
            biased(q + "q", l["heads"] * l["dim"], d)
            biased(q + "k", l["kv_heads"] * l["dim"], d)
            biased(q + "v", l["kv_heads"] * l["vdim"], d)
            biased(q + "o", d, l["heads"] * l["vdim"])
            out.update({q + "sink": (l["heads"],), q + "g": (l["heads"], d)})
            q, nk, nv = p + "mix.right.", r["heads"] * r["dim"], r["heads"] * r["vdim"]
            out.update({q + "q": (nk, d), q + "k": (nk, d), q + "v": (nv, d), q + "g": (nv, d), q + "o": (d, nv),
                        q + "norm": (r["vdim"],), q + "a1": (layer["_rank"], d)})
            biased(q + "a2", nk, layer["_rank"])
        if mlp is not None:
            out[p + "norm2"] = (d,)
            biased(p + "mlp.up", mlp["ff"], d)
            biased(p + "mlp.down", d, mlp["ff"])
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
        elif name == "embed" or last == "sink":
            pass
        elif last == "D":
            t = 1.0 + 0.5 * t
        elif last == "A_log":
            t = t - 1.0
        elif last == "dt_bias":
            t = t - 1.5
        elif last == "conv":
            t = t / math.sqrt(shape[1])
        elif name.endswith("a2.b"):
            t = 2.0 + t
        elif last == "b":
            t = 0.4 * t
        else:
            t = t / math.sqrt(shape[1])
            if name.endswith(("left.q", "left.k")):
                t = t * qk_gain
        out[name] = t.to(torch.bfloat16)
    return out
