"""Loader for the native engine extension (`aios_amd/_engine*.so`).

torch is imported first on purpose: torch-ROCm bundles `libamdhip64.so.7`; importing it before
the extension makes the dynamic loader resolve our DT_NEEDED entry to that same runtime, so one
process never holds two HIP runtimes.

On a machine with a GPU the extension is mandatory: `require()` raises instead of silently
falling back to a Python path (the round-end checks record which .so files were loaded).
"""
from __future__ import annotations

import importlib
import os
from typing import Optional

_mod = None
_err: Optional[BaseException] = None


def load(build_if_missing: bool = True, formats: str = "all"):
    """The extension with the kernels of every weight format; formats="bf16": also the smaller build of the
    bf16 kernels alone, which is what is compiled then if neither is there."""
    global _mod, _err
    if _mod is not None:
        return _mod
    try:
        import torch  # noqa: F401  (see module docstring)
    except Exception:  # pragma: no cover - torch is present in this image
        pass
    names = ["_engine"] + (["_engine_bf16"] if formats == "bf16" else [])
    for n in names:
        try:
            _mod = importlib.import_module("aios_amd." + n)
            return _mod
        except ImportError as e:
            _err = e
    if build_if_missing and os.environ.get("AIOS_NO_AUTOBUILD") != "1":
        from .. import _build

        _build.build(verbose=False, formats=formats)
        importlib.invalidate_caches()
        _mod = importlib.import_module("aios_amd." + names[-1])
        return _mod
    raise ImportError(f"aios_amd native engine not built: {_err}")


def available() -> bool:
    try:
        load(build_if_missing=False)
        return True
    except Exception:
        return False


def gpu_available() -> bool:
    try:
        import torch

        return torch.cuda.is_available() and torch.cuda.device_count() > 0
    except Exception:
        return False


def require(formats: str = "all"):
    """The native engine, loudly: on a GPU box a missing extension is an error."""
    return load(build_if_missing=True, formats=formats)


KV_DTYPES = ("bf16", "fp8", "fp8_e4m3")


def kv_fp8_flag(kv_dtype: str) -> int:
    """KV cache dtype name -> EngineConfig.kv_fp8: 'bf16' (default) or 'fp8' / 'fp8_e4m3' (OCP e4m3
    with per-layer K / V scales, half the cache bytes)."""
    k = (kv_dtype or "bf16").strip().lower()
    if k not in KV_DTYPES:
        raise ValueError(f"kv_dtype must be one of {KV_DTYPES}, not {kv_dtype!r}")
    return 0 if k == "bf16" else 1


def cu_mask_words(n: int, first: int = 0, total: int = 256) -> list:
    """A CU mask (32 CUs per word) of n CUs for one co-resident tier: CU slots [first, first + n/8) of
    every aligned group of 32 CU ids.  Whether the driver numbers CUs XCD-major (32 per XCD) or
    XCD-minor (id % 8), every XCD then keeps CUs of the tier (no XCD left without any -- each XCD has
    its own L2 and dispatcher) and two tiers with disjoint [first, first + n/8) ranges never share a CU.
    n must be a multiple of 8 between 64 and total."""
    if n % 8 or not (64 <= n <= total) or total % 32:
        raise ValueError(f"cu mask: {n} CUs (multiple of 8, 64..{total})")
    per = n // (total // 32)
    if first < 0 or first + per > 32:
        raise ValueError("cu mask: slot range outside the 32-CU group")
    words = [0] * (total // 32)
    for i in range(total):
        if first <= i % 32 < first + per:
            words[i // 32] |= 1 << (i % 32)
    return words


def engine_config(cfg, max_ctx: Optional[int] = None, max_slots: int = 4, max_batch: int = 8, device: int = 0,
                  tp_rank: int = 0, tp_size: int = 1, act_q8: bool = True, vocab_parallel: bool = True,
                  cu_mask: Optional[list] = None, kv_dtype: str = "bf16", compute: str = "bf16", kv_pool_tokens: int = 0):
    """aios_amd.models.config.ModelConfig -> native EngineConfig (per-rank shapes under TP).
    Under TP the lm_head is vocab-parallel (V/tp rows per rank + logits all-gather) unless the
    embeddings are tied or V is not divisible by tp.  compute "float32" (layered models): everything
    in 32 bits.  kv_pool_tokens: tokens the cache pool holds (0: every slot's full context)."""
    m = require()
    ec = m.EngineConfig()
    ec.name = cfg.name
    ec.vocab_size = cfg.vocab_size
    ec.d_model = cfg.d_model
    ec.n_layers = cfg.n_layers
    if cfg.n_heads % tp_size or cfg.n_kv_heads % tp_size or cfg.d_ff % tp_size:
        raise ValueError(f"TP={tp_size} does not divide heads/kv_heads/d_ff of {cfg.name}")
    ec.n_heads = cfg.n_heads // tp_size
    ec.n_kv_heads = cfg.n_kv_heads // tp_size
    ec.head_dim = cfg.head_dim
    ec.d_ff = cfg.d_ff // tp_size
    ec.rope_theta = float(cfg.rope_theta)
    ec.rope_neox = 1 if cfg.rope_mode == 2 else 0
    ec.norm_eps = float(cfg.norm_eps)
    ec.max_ctx = int(max_ctx or cfg.max_ctx)
    ec.max_slots = max_slots
    ec.max_batch = max_batch
    ec.tie_embeddings = int(cfg.tie_embeddings)
    ec.qk_norm = int(cfg.qk_norm)
    ec.qkv_bias = int(cfg.qkv_bias)
    ec.tp_rank = tp_rank
    ec.tp_size = tp_size
    ec.vocab_parallel = int(bool(vocab_parallel) and tp_size > 1 and not cfg.tie_embeddings
                            and cfg.vocab_size % tp_size == 0)
    ec.device = device
    if cu_mask:
        ec.cu_mask = [int(w) & 0xFFFFFFFF for w in cu_mask]
    ec.kv_fp8 = kv_fp8_flag(kv_dtype)
    ec.act_q8 = int(act_q8)
    ec.kv_pool_tokens = int(kv_pool_tokens)
    if compute not in ("bf16", "bfloat16", "f32", "float32"):
        raise ValueError(f"compute must be bfloat16 or float32, not {compute!r}")
    ec.compute_f32 = int(compute in ("f32", "float32"))
    if ec.compute_f32 and not cfg.layers:
        raise ValueError(f"{cfg.name}: only layered models compute in 32 bits")
    if cfg.layers:
        if tp_size > 1:
            raise ValueError(f"{cfg.name}: layered models run on one GPU (no tensor parallelism)")
        if ec.kv_fp8:
            raise ValueError(f"{cfg.name}: the cache has no fp8 form (kv_dtype bf16)")
        ec.max_positions = int(cfg.max_ctx) if cfg.learned_pos else 0
        ec.embed_scale, ec.logit_scale = float(cfg.embed_scale), float(cfg.logit_scale)
        if cfg.bigram:
            ec.bigram_buckets, ec.bigram_prev, ec.bigram_cur = (int(v) for v in cfg.bigram)
        if cfg.loop:
            ec.loop_start, ec.loop_stop, ec.loop_times = (int(v) for v in cfg.loop)
            ec.loop_add = int(cfg.loop_add)
        ec.layers = [_layer_spec(m, l) for l in cfg.layers]
    return ec


def _layer_spec(m, l):
    s = m.LayerSpec()
    kinds = {"": m.MIX_NONE, "latent": m.MIX_LATENT, "mingru": m.MIX_MINGRU, "gqa": m.MIX_GQA, "mamba2": m.MIX_MAMBA2,
             "gla": m.MIX_GLA, "delta": m.MIX_DELTA}
    s.mixer, s.beside = kinds[l.mixer], kinds[l.beside]
    s.mixer_scale, s.beside_scale = float(l.mixer_scale), float(l.beside_scale)
    s.kv_heads, s.chunk, s.softcap, s.attn_bias = l.kv_heads, l.chunk, float(l.softcap), (1 if l.out_bias else 2) if l.attn_bias else 0
    s.qk_norm, s.v_norm, s.head_temp, s.v_mix = int(l.qk_norm), int(l.v_norm), int(l.head_temp), int(l.v_mix)
    if l.lin is not None:
        lin = m.LinSpec()
        lin.heads, lin.groups, lin.dim, lin.vdim = l.lin.heads, l.lin.groups, l.lin.dim, l.lin.vdim
        lin.conv, lin.norm_groups, lin.rank, lin.tau = l.lin.conv, l.lin.norm_groups, l.lin.rank, float(l.lin.tau)
        s.lin = lin
    s.parallel, s.norm_scalar = int(l.parallel), int(l.norm_scalar)
    s.post_norm, s.resid_gate = int(l.post_norm), int(l.resid_gate)
    s.heads, s.dim, s.vdim, s.kv_rank = l.heads, l.dim, l.vdim, l.kv_rank
    s.rot_dim, s.rot_dims, s.rot_base, s.window = l.rot_dim, l.rot_dims, float(l.rot_base), l.window
    s.scale = float(l.scale)
    s.sink = 2 if l.sink_one else int(l.sink)
    s.out_gate = {"none": m.GATE_NONE, "element": m.GATE_ELEMENT, "head": m.GATE_HEAD}[l.out_gate]
    s.width = l.width
    s.mlp, s.ff = (m.MLP_MOE if l.experts else m.MLP_GLU if l.gated else m.MLP_ACT, l.ff) if l.ff else (m.MLP_NONE, 0)
    s.act = {"gelu_tanh": m.ACT_GELU_TANH, "silu": m.ACT_SILU, "relu2": m.ACT_RELU2,
             "xielu": m.ACT_XIELU}[l.act]
    if s.mlp in (m.MLP_GLU, m.MLP_MOE) and s.act in (m.ACT_RELU2, m.ACT_XIELU):
        raise ValueError(f"{l.act} is no gate's activation")
    s.mlp_bias, s.mlp_scale = int(l.mlp_bias), float(l.mlp_scale)
    s.experts, s.top, s.shared_ff = l.experts, l.top, l.shared_ff
    s.router_scale, s.correction = float(l.router_scale), int(l.correction)
    s.weights_of = l.weights_of
    return s
