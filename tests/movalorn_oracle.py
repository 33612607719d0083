"""Plain, slow oracle of the Movalorn decoder for the tests: one function per mechanism, whole sequences at
once, no cache, no state between calls, no batching, no page, no fused, absorbed or chunked form, float64 by
default.  Shares nothing with aios_amd: it takes the parsed config.json and a {tensor name: tensor} dict.

Notation: t, s positions; h a head; r the latent width; x the residual stream [T, width].
"""
from __future__ import annotations

import math
from typing import Dict, List, Optional

import torch

DT = torch.float64


# ---- mechanisms ----------------------------------------------------------------------------------
def rms(x: torch.Tensor, eps: float) -> torch.Tensor:
    return x / torch.sqrt(x.pow(2).mean(-1, keepdim=True) + eps)


def scalar_norm(x: torch.Tensor, g: torch.Tensor, eps: float) -> torch.Tensor:
    """RMS norm with one gain for all coordinates."""
    return rms(x, eps) * g.reshape(())


def gelu_tanh(z: torch.Tensor) -> torch.Tensor:
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def silu(z: torch.Tensor) -> torch.Tensor:
    return z * torch.sigmoid(z)


def bigram_rows(tokens: List[int], mul_prev: int, mul_cur: int, buckets: int) -> List[int]:
    """Row of the pair table per token; the row after the last bucket where there is no token before."""
    return [buckets if t == 0 else (tokens[t - 1] * mul_prev + tokens[t] * mul_cur) % buckets
            for t in range(len(tokens))]


def embed(tokens: List[int], w: Dict[str, torch.Tensor], e: dict) -> torch.Tensor:
    b = e["bigram"]
    rows = bigram_rows(tokens, b["mul_prev"], b["mul_cur"], b["buckets"])
    return torch.stack([w["embed"][t] * e["scale"] + w["bigram"][r] for t, r in zip(tokens, rows)])


def rotate(v: torch.Tensor, base: float, dims: int) -> torch.Tensor:
    """v [T, ..., n] with row t at position t: pairs (2i, 2i+1), i < dims / 2, turned by t base^(-2i/dims)."""
    out = v.clone()
    T = v.shape[0]
    for i in range(dims // 2):
        a = torch.arange(T, dtype=v.dtype) * base ** (-2.0 * i / dims)
        a = a.reshape([T] + [1] * (v.dim() - 2))
        x, y = v[..., 2 * i], v[..., 2 * i + 1]
        out[..., 2 * i] = x * torch.cos(a) - y * torch.sin(a)
        out[..., 2 * i + 1] = y * torch.cos(a) + x * torch.sin(a)
    return out


def latent(h: torch.Tensor, w: Dict[str, torch.Tensor], p: str, m: dict, eps: float):
    """What a token leaves for later ones: its normalised latent, and the rotated key part all heads share."""
    y = h @ w[p + "dkv"].T
    c = rms(y[:, :m["kv_rank"]], eps) * w[p + "dkv.norm"]
    return c, rotate(y[:, m["kv_rank"]:], m["rot"]["base"], m["rot"]["dims"])


def visible(i: int, size: int) -> range:
    """Keys of query i under a window of `size` tokens, itself included."""
    return range(max(0, i - size + 1), i + 1)


def latent_attention(h: torch.Tensor, w: Dict[str, torch.Tensor], p: str, m: dict, eps: float) -> torch.Tensor:
    T, H, dk, dr, dv = h.shape[0], m["heads"], m["dim"], m["rot_dim"], m["vdim"]
    q = (h @ w[p + "q"].T).view(T, H, dk + dr)
    qu, qr = q[..., :dk], rotate(q[..., dk:], m["rot"]["base"], m["rot"]["dims"])
    c, kr = latent(h, w, p, m, eps)
    ku = (c @ w[p + "uk"].T).view(T, H, dk)
    v = (c @ w[p + "uv"].T).view(T, H, dv)
    out = torch.zeros(T, H, dv, dtype=h.dtype)
    for i in range(T):
        see = visible(i, m["mask"]["size"])
        a, b = see.start, see.stop
        for n in range(H):
            score = (ku[a:b, n] @ qu[i, n] + kr[a:b] @ qr[i, n]) * m["scale"]
            out[i, n] = torch.softmax(score, 0) @ v[a:b, n]
    out = out * torch.sigmoid(h @ w[p + "g"].T)[..., None]
    return out.reshape(T, H * dv) @ w[p + "o"].T


def mingru_states(z: torch.Tensor, u: torch.Tensor, s0: Optional[torch.Tensor] = None) -> torch.Tensor:
    """S_t = (1 - sig(z_t)) S_{t-1} + sig(z_t) cand(u_t), cand(u) = u + 1/2 for u >= 0, sig(u) below."""
    s = torch.zeros_like(u[0]) if s0 is None else s0
    out = []
    for t in range(u.shape[0]):
        f = torch.sigmoid(z[t])
        cand = torch.where(u[t] >= 0, u[t] + 0.5, torch.sigmoid(u[t]))
        s = (1 - f) * s + f * cand
        out.append(s)
    return torch.stack(out)


def mingru(h: torch.Tensor, w: Dict[str, torch.Tensor], p: str) -> torch.Tensor:
    s = mingru_states(h @ w[p + "z"].T + w[p + "z.b"], h @ w[p + "x"].T + w[p + "x.b"])
    return (s * silu(h @ w[p + "g"].T)) @ w[p + "o"].T


def glu(h: torch.Tensor, w: Dict[str, torch.Tensor], p: str, act) -> torch.Tensor:
    return (act(h @ w[p + "gate"].T) * (h @ w[p + "up"].T)) @ w[p + "down"].T


def route(h: torch.Tensor, w: Dict[str, torch.Tensor], p: str, r: dict):
    """(experts [T, top], their weights): chosen by score + correction, weighted by the score alone."""
    s = torch.softmax(h @ w[p + "router"].T, -1)
    pick = torch.topk(s + w[p + "correction"], r["top"], -1).indices
    return pick, torch.gather(s, 1, pick) * r["scale"]


def choice_gap(h: torch.Tensor, w: Dict[str, torch.Tensor], p: str, r: dict) -> torch.Tensor:
    """How far the last chosen expert's choice score is above the first one left out [T]."""
    if r["top"] == r["experts"]:
        return torch.ones(h.shape[0], dtype=h.dtype)
    c = torch.sort(torch.softmax(h @ w[p + "router"].T, -1) + w[p + "correction"], -1, descending=True).values
    return c[:, r["top"] - 1] - c[:, r["top"]]


def moe(h: torch.Tensor, w: Dict[str, torch.Tensor], p: str, m: dict) -> torch.Tensor:
    pick, wt = route(h, w, p, m["router"])
    y = torch.zeros_like(h)
    for e in range(m["router"]["experts"]):
        for k in range(m["router"]["top"]):
            on = pick[:, k] == e
            if bool(on.any()):
                y[on] += wt[on, k, None] * glu(h[on], w, f"{p}e{e}.", silu)
    if m.get("shared"):
        y = y + glu(h, w, p + "shared.", silu)
    return y


def feed_forward(h: torch.Tensor, w: Dict[str, torch.Tensor], p: str, m: dict) -> torch.Tensor:
    return glu(h, w, p, gelu_tanh) if m["kind"] == "dense" else moe(h, w, p, m)


def sublayer(x: torch.Tensor, w: Dict[str, torch.Tensor], p: str, n: int, eps: float, f) -> torch.Tensor:
    """x + norm_b( f(h) * sigmoid(gate h) ), h = norm(x)."""
    h = scalar_norm(x, w[f"{p}norm{n}"], eps)
    y = f(h) * torch.sigmoid(h @ w[f"{p}rg{n}"].T + w[f"{p}rg{n}.b"])
    return x + scalar_norm(y, w[f"{p}norm{n}b"], eps)


def schedule(cfg: dict) -> List[tuple]:
    """(layer, pass) in running order; pass -1 outside the loop."""
    n, lp = len(cfg["layers"]), cfg.get("loop")
    if not lp:
        return [(i, -1) for i in range(n)]
    return ([(i, -1) for i in range(lp["start"])] +
            [(i, t) for t in range(lp["times"]) for i in range(lp["start"], lp["stop"])] +
            [(i, -1) for i in range(lp["stop"], n)])


def forward(cfg: dict, w: Dict[str, torch.Tensor], tokens: List[int], trace: Optional[list] = None,
            dtype=DT, gaps: Optional[list] = None) -> torch.Tensor:
    """Logits [T, vocab]; `trace` collects the residual stream after every layer run, `gaps` the experts' choice
    gaps of every layer run that has a router."""
    w = {k: v.to(dtype) for k, v in w.items()}
    eps = cfg["norm"]["eps"]
    x = x0 = embed(tokens, w, cfg["embedding"])
    for i, t in schedule(cfg):
        if t >= 0 and i == cfg["loop"]["start"]:
            x = torch.cat([x, x0], -1) @ w["loop.in"].T + w["loop.step"][t]
        layer, p = cfg["layers"][i], f"l{i}."
        if layer["type"] == "mingru":
            mix = lambda h: mingru(h, w, p + "mix.")
        else:
            mix = lambda h: latent_attention(h, w, p + "mix.", layer["mixer"], eps)
        x = sublayer(x, w, p, 1, eps, mix)
        if layer.get("mlp") is not None:
            if gaps is not None and layer["mlp"]["kind"] == "moe":
                gaps.append(choice_gap(scalar_norm(x, w[p + "norm2"], eps), w, p + "mlp.", layer["mlp"]["router"]))
            x = sublayer(x, w, p, 2, eps, lambda h: feed_forward(h, w, p + "mlp.", layer["mlp"]))
        if trace is not None:
            trace.append(x)
    return scalar_norm(x, w["final.norm"], eps) @ w["head"].T * cfg["logit_scale"]


def greedy(cfg: dict, w: Dict[str, torch.Tensor], prompt: List[int], n: int) -> List[int]:
    ids = list(prompt)
    for _ in range(n):
        ids.append(int(forward(cfg, w, ids)[-1].argmax()))
    return ids[len(prompt):]


# ---- random models of any size ------------------------------------------------------------------
def make_config(width=96, vocab=211, eps=3e-5, layers=None, loop=None, scale=0.8, bigram=(101, 7, 3),
                logit_scale=0.6) -> dict:
    return {"architecture": "Movalorn", "width": width, "vocab": vocab, "norm": {"eps": eps},
            "embedding": {"scale": scale, "bigram": dict(zip(("buckets", "mul_prev", "mul_cur"), bigram))},
            "loop": None if loop is None else dict(zip(("start", "stop", "times"), loop)), "layers": layers,
            "logit_scale": logit_scale}


def dense(ff: int) -> dict:
    return {"kind": "dense", "ff": ff}


def experts(n: int, top: int, ff: int, shared: Optional[int], scale=1.3) -> dict:
    m = {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": n, "top": top, "scale": scale}}
    return dict(m, shared={"ff": shared}) if shared else m


def attention_layer(mlp, heads=3, dim=24, rot_dim=8, vdim=40, kv_rank=56, scale=0.17, window=17, base=3000.0) -> dict:
    return {"type": "latent_attention", "mlp": mlp,
            "mixer": {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank, "scale": scale,
                      "mask": {"size": window}, "rot": {"base": base, "dims": rot_dim}}}


def gru_layer(mlp, width=80) -> dict:
    return {"type": "mingru", "mlp": mlp, "mixer": {"width": width}}


def tensor_shapes(cfg: dict) -> Dict[str, tuple]:
    d, V = cfg["width"], cfg["vocab"]
    out = {"embed": (V, d), "bigram": (cfg["embedding"]["bigram"]["buckets"] + 1, d), "final.norm": (), "head": (V, d)}
    if cfg.get("loop"):
        out.update({"loop.in": (d, 2 * d), "loop.step": (cfg["loop"]["times"], d)})

    def ffn(p, ff):
        out.update({p + "gate": (ff, d), p + "up": (ff, d), p + "down": (d, ff)})

    for i, layer in enumerate(cfg["layers"]):
        m, p, mlp = layer["mixer"], f"l{i}.", layer.get("mlp")
        for n in (1, 2) if mlp is not None else (1,):
            out.update({f"{p}norm{n}": (), f"{p}norm{n}b": (), f"{p}rg{n}": (d, d), f"{p}rg{n}.b": (d,)})
        if layer["type"] == "mingru":
            n = m["width"]
            out.update({p + "mix.z": (n, d), p + "mix.z.b": (n,), p + "mix.x": (n, d), p + "mix.x.b": (n,),
                        p + "mix.g": (n, d), p + "mix.o": (d, n)})
        else:
            H, dk, dr, dv, r = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
            out.update({p + "mix.q": (H * (dk + dr), d), p + "mix.dkv": (r + dr, d), p + "mix.dkv.norm": (r,),
                        p + "mix.uk": (H * dk, r), p + "mix.uv": (H * dv, r), p + "mix.g": (H, d),
                        p + "mix.o": (d, H * dv)})
        if mlp is None:
            continue
        if mlp["kind"] == "dense":
            ffn(p + "mlp.", mlp["ff"])
            continue
        E = mlp["router"]["experts"]
        out.update({p + "mlp.router": (E, d), p + "mlp.correction": (E,)})
        for e in range(E):
            ffn(f"{p}mlp.e{e}.", mlp["expert"]["ff"])
        if mlp.get("shared"):
            ffn(p + "mlp.shared.", mlp["shared"]["ff"])
    return out


def random_weights(cfg: dict, seed: int = 0, qk_gain: float = 1.0, classes: int = 0) -> Dict[str, torch.Tensor]:
    """bf16 weights; qk_gain > 1 sharpens the attention (single keys stand out).  classes > 0: a token's class
    (token mod classes) stands in columns of its own through all layers, and the routers go mostly by it, so that
    hardly any choice of experts is close."""
    g = torch.Generator().manual_seed(seed)
    out = {}
    for name, shape in tensor_shapes(cfg).items():
        t = torch.randn(shape, generator=g, dtype=torch.float32)
        if name.split(".")[-1].startswith("norm"):
            t = 1.0 + 0.3 * t
        elif name in ("embed", "bigram"):
            t = t * (1.0 if name == "embed" else 0.7)
        elif name.endswith(".b"):
            t = t * 0.7
        elif name.endswith("correction"):
            t = t * 0.2
        elif name.endswith("router"):
            t = t * 2 / math.sqrt(shape[1])
        elif name == "loop.step":
            t = t * 0.5
        else:
            t = t / math.sqrt(shape[1])
            if name.endswith((".q", ".uk", ".dkv")):
                t = t * qk_gain
        if classes:
            if name in ("embed", "bigram", "loop.step"):
                t[:, :classes] = 0
            if name == "embed":
                for c in range(classes):
                    t[c::classes, c] = 8.0
            elif name.endswith((".o", ".down", "loop.in")):
                t[:classes] = 0
                if name == "loop.in":
                    t[:classes, shape[0]:shape[0] + classes] = torch.eye(classes)
            elif name.endswith("router"):
                t *= 0.05
                for c in range(classes):
                    t[:, c] = torch.linspace(-1, 1, shape[0])[torch.randperm(shape[0], generator=g)]
        out[name] = t.to(torch.bfloat16)
    return out
