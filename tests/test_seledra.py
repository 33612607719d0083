"""Seledra on the CPU: configuration, registry, presets, and the oracle the GPU tests compare against -- including that
each mechanism, left out or shifted by one, would show in the logits those tests look at."""
import asyncio
import math

import numpy as np
import pytest
import torch

import seledra_oracle as O
from aios_amd.models import registry
from aios_amd.models.config import LayerConfig, LinConfig, get_preset
from test_gefazen import rel, write_model

# unlike sizes everywhere; layers with and without an MLP; values mixed by some attention layers, whose first is not the
# model's first; heads that share one key head, or have one each; odd sizes and taps
MIXED = O.make_config(layers=[
    O.delta_layer(O.dense(72)),
    O.attn_layer(None, heads=4, kv_heads=1, dim=24, vdim=40, scale=0.27, v_mix=False),
    O.attn_layer(O.dense(40)),
    O.delta_layer(None, heads=5, kv_heads=5, dim=33, vdim=10, conv=2),
    O.attn_layer(None, heads=9, kv_heads=3, dim=14, vdim=28, scale=0.35),
    O.delta_layer(O.dense(50), heads=3, kv_heads=1, dim=40, vdim=17, conv=5),
    O.attn_layer(O.dense(33), heads=3, kv_heads=3, dim=32, vdim=28, scale=0.2)])


def ids_of(n, seed=0, vocab=211):
    return [int(t) for t in np.random.default_rng(seed).integers(0, vocab, n)]


# ---- configuration and checkpoints -----------------------------------------------------------------
def test_config_reads_every_size_and_branch(tmp_path):
    path = write_model(tmp_path / "m", MIXED, O.random_weights(MIXED))
    cfg, raw, arch = registry.load_config(path)
    assert (cfg.vocab_size, cfg.d_model, cfg.norm_eps, cfg.n_layers, cfg.learned_pos, cfg.max_ctx) == (211, 96, 3e-5, 7, True, 300)
    assert (cfg.loop, cfg.embed_scale, cfg.logit_scale, cfg.bigram) == (None, 1.0, 1.0, None)
    common = dict(parallel=False, gated=False, act="xielu", mixer_scale=0.8, mlp_scale=0.8, sink=False)
    att = dict(mixer="gqa", sink_one=True, out_gate="head", attn_bias=True, out_bias=False, qk_norm=True, v_norm=True,
               head_temp=True, **common)
    assert cfg.layers[0] == LayerConfig(mixer="delta", out_gate="none", ff=72, **common,
                                        lin=LinConfig(heads=6, groups=2, dim=24, vdim=20, conv=4))
    assert cfg.layers[1] == LayerConfig(heads=4, kv_heads=1, dim=24, vdim=40, scale=0.27, v_mix=False, ff=0, **att)
    assert cfg.layers[2] == LayerConfig(heads=6, kv_heads=3, dim=20, vdim=28, scale=0.3, v_mix=True, ff=40, **att)
    assert cfg.layers[3].lin.conv == 2 and cfg.layers[3].ff == 0 and cfg.layers[6].ff == 33
    names = arch.tensor_names(raw)
    assert set(names) == set(O.tensor_shapes(MIXED)) and len(set(names.values())) == len(names)
    assert "l1.mix.vmix" not in names and names["l2.mix.vmix"] == "blk.2.attn_v_mix.weight" and "l3.norm2" not in names
    assert registry.is_checkpoint_dir(path)
    assert cfg.n_params() == pytest.approx(sum(math.prod(s) for s in O.tensor_shapes(MIXED).values()), rel=0.02)


@pytest.mark.parametrize("layers, message", [
    ([dict(O.delta_layer(None), type="other")], "mixer type"),
    ([dict(O.delta_layer(None), mlp={"kind": "sparse", "ff": 8})], "feed-forward"),
    ([O.delta_layer(None, heads=5, kv_heads=2)], "key heads"), ([O.attn_layer(None, heads=4, kv_heads=3)], "key heads"),
    ([O.attn_layer(None), O.attn_layer(None, vdim=24)], "value heads")])
def test_config_rejects_what_does_not_fit(layers, message):
    with pytest.raises(ValueError, match=message):
        registry.get("Seledra").parse(O.make_config(layers=layers), "m")


def test_presets_name_the_design():
    for name in ("seledra-1b", "seledra-7b", "test-seledra"):
        cfg = get_preset(name)
        assert cfg.arch == "seledra" and len(cfg.layers) == cfg.n_layers and cfg.n_params() > 0
        assert {l.mixer for l in cfg.layers} == {"gqa", "delta"}


def test_cpu_backend_refuses_layered_models(tmp_path):
    from aios_amd.runtime.model_manager import ModelManager

    folder = write_model(tmp_path / "m", MIXED, O.random_weights(MIXED))
    m = asyncio.run(ModelManager(max_batch=2, max_slots=2).load_model("seledra-cpu", folder + "#cpu"))
    assert m.status != "ready" and m.error


# ---- oracle ----------------------------------------------------------------------------------------
def test_oracle_mechanisms_by_hand():
    t = lambda *v: torch.tensor(v, dtype=O.DT)
    assert torch.allclose(O.rms(t([3.0, -4.0], [1.0, 1.0]), 0.5), t([3 / math.sqrt(13), -4 / math.sqrt(13)], [1 / math.sqrt(1.5)] * 2))
    assert torch.allclose(O.softplus(t(-800.0, 0.0, 3.0, 800.0)), t(0.0, math.log(2), math.log1p(math.exp(3)), 800.0))
    p, q = t(0.3), t(-0.7)
    sp, sq = math.log1p(math.exp(0.3)), math.log1p(math.exp(-0.7))
    assert torch.allclose(O.xielu(t(2.0, 0.0, -3.0), p, q), t(4 * sp + 1, 0.0, (0.5 + sq) * (math.exp(-3) + 2) - 1.5))
    assert torch.allclose(O.weights(t(0.0, math.log(3))), t(1 / 5, 3 / 5))
    assert torch.allclose(O.scores(t(1.0, 2.0), t([3.0, 4.0]), 0.5, t(2.0)), t(11.0))
    assert torch.allclose(O.mix_values(t(4.0), t(8.0), t(0.25)), t(5.0))
    assert torch.allclose(O.unit(t([3.0, 4.0])), t([0.6, 0.8]))
    assert torch.allclose(O.decay(t(1.0), t(0.0), t(2.0)), torch.exp(-O.softplus(t(3.0))))
    u = torch.arange(4, dtype=O.DT)[:, None] + 1
    assert torch.allclose(O.causal_conv(u, t([5.0, 7.0, 11.0]))[:, 0], t(11, 22 + 7, 33 + 14 + 5, 44 + 21 + 10))
    # two tokens, one head, one row and column: S1 = k b v; S2 = g S1 + k2 b2 (v2 - g S1 k2)
    g, b = t([0.9], [0.5]), t([0.8], [0.4])
    k, v, q = (x[:, None, None] for x in (t(0.6, -0.8), t(2.0, 3.0), t(1.0, 4.0)))
    s1 = 0.6 * 0.8 * 2
    s2 = 0.5 * s1 - 0.8 * 0.4 * (3 + 0.5 * s1 * 0.8)
    assert torch.allclose(O.delta_rule(g, b, k, v, q).flatten(), t(s1, 4 * s2))
    # a strength of 1 and no decay: reading with the key that was just written gives the value
    k = O.unit(torch.randn(5, 1, 3, dtype=O.DT, generator=torch.Generator().manual_seed(1)))
    v = torch.randn(5, 1, 2, dtype=O.DT, generator=torch.Generator().manual_seed(2))
    assert torch.allclose(O.delta_rule(torch.ones(5, 1).double(), torch.ones(5, 1).double(), k, v, k), v, atol=1e-4)
    w, ids = O.random_weights(MIXED, 3), ids_of(20)
    assert torch.allclose(O.forward(MIXED, w, ids)[:9], O.forward(MIXED, w, ids[:9]))  # causal


FAULTS = ["no position", "position shifted", "q norm per head", "k norm per head", "norm weights", "one-plus norm", "no value norm",
          "value norm over all", "no temp", "temp per key head", "scale", "learned sink", "no sink", "q bias", "k bias", "v bias",
          "wrong key head", "values not mixed", "mixed the other way", "first mixed with zeros", "mixed with the one before",
          "mixed where not asked", "no gate per head", "gate of another head", "taps reversed", "conv lost", "no silu after the conv",
          "conv of v left out", "no unit q", "no unit k", "q scale", "state lost", "decay", "decay after the write", "no decay in the read",
          "no strength", "strength shifted", "read before the write", "no delta", "wrong group", "no step bias", "delta norm per row",
          "delta norm weight", "delta gate", "xielu numbers swapped", "xielu below zero", "residual scale", "residual scale of the mlp",
          "final norm"]


@pytest.mark.parametrize("fault", FAULTS)
def test_a_fault_in_any_mechanism_shows(fault, monkeypatch):
    """Planted in the oracle: some logits move by far more than the GPU tests' tolerances (7e-2 in bf16)."""
    cfg, w = MIXED, O.random_weights(MIXED, 1, qk_gain=3.0)
    ids = ids_of(40, 1)
    over = lambda f, *ends: {k: (f(v) if k.endswith(ends) else v) for k, v in w.items()}
    # numbers with which the fault is large enough to show
    if fault in ("k bias", "q bias"):
        w = over(lambda v: v * 4, "mix.k.b", "mix.q.b")
    elif "temp" in fault:
        w = over(lambda v: 1 + 4 * (v - 1), ".temp")
    elif fault in ("q norm per head", "value norm over all"):  # (heads of unlike size)
        grow = lambda v: v * torch.linspace(0.3, 3.0, v.shape[0]).reshape((-1,) + (1,) * (v.dim() - 1))
        w = over(grow, "mix.q", "mix.v", "mix.v.b")
    elif fault in ("q scale", "no unit q"):  # (shows through the norm's eps alone)
        cfg = dict(cfg, norm={"eps": 0.02})
    elif "decay" in fault or fault in ("read before the write", "no delta"):
        w = over(lambda v: v + 1.5, "dt_bias")
    good = O.forward(cfg, w, ids)
    zero = lambda *ends: over(torch.zeros_like, *ends)
    real = {n: getattr(O, n) for n in ("rms", "whole_norm", "value_norm", "mix_values", "attention", "causal_conv", "unit", "decay",
                                       "delta_rule", "delta", "silu", "xielu", "feed_forward")}
    patch = lambda n, f: monkeypatch.setattr(O, n, f)
    cut = lambda f: (lambda *a: torch.cat([f(*(x[:30] for x in a)), f(*(x[30:] for x in a))]))

    def rule(form):
        def f(g, beta, k, v, q):
            S = torch.zeros(k.shape[1], k.shape[2], v.shape[2], dtype=v.dtype)
            out = []
            for t in range(v.shape[0]):
                G, dot = g[t][:, None, None], lambda s, x: (s * x[t][:, :, None]).sum(1)
                u = beta[t][:, None] * (v[t] - dot(S if form == "read" else G * S, k))
                if form == "none":
                    u = beta[t][:, None] * v[t]
                w = k[t][:, :, None] * u[:, None, :]
                old, S = G * S, G * (S + w) if form == "after" else G * S + w
                out.append(dot(old if form == "early" else S, q))
            return torch.stack(out)
        return f

    if fault in ("no temp", "no step bias", "no gate per head", "q bias", "k bias", "v bias", "delta norm weight", "norm weights"):
        w = {"no temp": lambda: over(torch.ones_like, ".temp"), "no step bias": lambda: zero("dt_bias"),
             "no gate per head": lambda: {k: torch.zeros_like(v) if k.endswith(".g") and v.shape[0] < 10 else v for k, v in w.items()},
             "q bias": lambda: zero(".q.b"), "k bias": lambda: zero(".k.b"), "v bias": lambda: zero(".v.b"),
             "delta norm weight": lambda: over(torch.ones_like, "mix.norm"),
             "norm weights": lambda: over(torch.ones_like, "q.norm", "k.norm")}[fault]()
    elif fault == "no position":
        w = zero("pos")
    elif fault == "position shifted":
        w = dict(w, pos=w["pos"].roll(1, 0))
    elif fault in ("q norm per head", "k norm per head"):
        def norm(y, g, eps):  # (queries are the wider of a layer's two, or the first)
            norm.n += 1
            if (norm.n % 2 == 1) != (fault[0] == "q"):
                return real["whole_norm"](y, g, eps)
            return real["rms"](y.view(y.shape[0], 2 if y.shape[1] % 3 else 3, -1), eps).reshape(y.shape) * g
        norm.n = 0
        patch("whole_norm", norm)
    elif fault == "one-plus norm":
        patch("whole_norm", lambda y, g, eps: real["whole_norm"](y, 1 + g, eps))
    elif fault == "no value norm":
        patch("value_norm", lambda v, eps: v)
    elif fault == "value norm over all":
        patch("value_norm", lambda v, eps: real["rms"](v.flatten(1), eps).view(v.shape))
    elif fault == "temp per key head":
        w = over(lambda v: v[:1].expand(v.shape), ".temp")
    elif fault == "scale":
        cfg = dict(cfg, layers=[dict(l, mixer=dict(l["mixer"], scale=l["mixer"]["dim"] ** -1.0)) if l["type"] == "attention" else l
                                for l in cfg["layers"]])
    elif fault == "learned sink":
        patch("weights", lambda s: torch.softmax(torch.cat([s, s.new_full((1,), 2.0)]), 0)[:-1])
    elif fault == "no sink":
        patch("weights", lambda s: torch.softmax(s, 0))
    elif fault == "wrong key head":
        w = over(lambda v: v.roll(v.shape[0] // 3, 0) if v.shape[0] % 3 == 0 else v, "mix.k")
    elif fault == "values not mixed":
        patch("mix_values", lambda v, f, l: v)
    elif fault == "mixed the other way":
        patch("mix_values", lambda v, f, l: real["mix_values"](f, v, l + 0.2))
    elif fault == "first mixed with zeros":
        def att(h, w, p, m, eps, shared):
            if not m["v_mix"] or "values" in shared:
                return real["attention"](h, w, p, m, eps, shared)
            with monkeypatch.context() as mp:
                seen = []
                mp.setattr(O, "value_norm", lambda v, e: (seen.append(real["rms"](v, e)), (1 - w[p + "vmix"]) * seen[0])[1])
                y = real["attention"](h, w, p, m, eps, shared)
            shared["values"] = seen[0]
            return y
        monkeypatch.setitem(O.MIXERS, "attention", att)
    elif fault == "mixed with the one before":
        def att(h, w, p, m, eps, shared):
            with monkeypatch.context() as mp:
                seen = []
                mp.setattr(O, "value_norm", lambda v, e: (seen.append(real["rms"](v, e)), seen[0])[1])
                y = real["attention"](h, w, p, m, eps, shared)
            if m["v_mix"]:
                shared["values"] = seen[0]
            return y
        monkeypatch.setitem(O.MIXERS, "attention", att)
    elif fault == "mixed where not asked":
        cfg = dict(cfg, layers=[dict(l, mixer=dict(l["mixer"], v_mix=True, kv_heads=1)) if i == 1 else
                                dict(l, mixer=dict(l["mixer"], v_mix=False)) if l["type"] == "attention" else l
                                for i, l in enumerate(cfg["layers"])])
        w = dict(w, **{"l1.mix.vmix": torch.tensor(0.5)})
    elif fault == "gate of another head":
        def att(h, w, p, m, eps, shared):
            return real["attention"](h, dict(w, **{p + "g": w[p + "g"].roll(1, 0)}), p, m, eps, shared)
        monkeypatch.setitem(O.MIXERS, "attention", att)
    elif fault == "taps reversed":
        w = over(lambda v: v.flip(1), ".conv")
    elif fault == "conv lost":  # a portion that starts without its predecessor's last inputs
        patch("causal_conv", lambda u, k: torch.cat([real["causal_conv"](u[:30], k), real["causal_conv"](u[30:], k)]))
    elif fault == "no silu after the conv":  # (the fourth of a layer's is the output gate's)
        def silu(z):
            silu.n += 1
            return real["silu"](z) if silu.n % 4 == 0 else z
        silu.n = 0
        patch("silu", silu)
    elif fault == "conv of v left out":
        w = over(lambda v: torch.cat([torch.zeros_like(v[:, :-1]), torch.ones_like(v[:, -1:])], 1), "v.conv")
    elif fault in ("no unit q", "no unit k"):
        def unit(x):
            unit.n += 1
            return x if (unit.n % 2 == 1) == (fault[-1] == "q") else real["unit"](x)
        unit.n = 0
        patch("unit", unit)
    elif fault == "q scale":
        patch("delta_rule", lambda g, b, k, v, q: real["delta_rule"](g, b, k, v, q * math.sqrt(q.shape[-1])))
    elif fault == "state lost":
        patch("delta_rule", cut(real["delta_rule"]))
    elif fault == "decay":
        patch("decay", lambda *a: real["decay"](*a).roll(1, 0))
    elif fault in ("decay after the write", "no decay in the read", "read before the write", "no delta"):
        patch("delta_rule", rule({"decay after the write": "after", "no decay in the read": "read", "read before the write": "early",
                                  "no delta": "none"}[fault]))
    elif fault == "no strength":
        patch("delta_rule", lambda g, b, k, v, q: real["delta_rule"](g, torch.ones_like(b), k, v, q))
    elif fault == "strength shifted":
        patch("delta_rule", lambda g, b, k, v, q: real["delta_rule"](g, b.roll(1, 0), k, v, q))
    elif fault == "wrong group":
        patch("delta_rule", lambda g, b, k, v, q: real["delta_rule"](g, b, k.roll(1, 1), v, q))
    elif fault == "delta norm per row":
        def mixer(h, w, p, m, eps, shared):
            with monkeypatch.context() as mp:
                mp.setattr(O, "rms", lambda x, e: real["rms"](x.flatten(1), e).view(x.shape))
                return real["delta"](h, w, p, m, eps, shared)
        monkeypatch.setitem(O.MIXERS, "delta", mixer)
    elif fault == "delta gate":
        w = {k: -v if k.endswith(".g") and v.shape[0] > 40 else v for k, v in w.items()}
    elif fault == "xielu numbers swapped":
        patch("xielu", lambda z, p, q: real["xielu"](z, q, p))
    elif fault == "xielu below zero":
        patch("xielu", lambda z, p, q: torch.where(z > 0, real["xielu"](z, p, q), z / 2))
    elif fault == "residual scale":
        cfg = dict(cfg, residual_mult=1.0)
    elif fault == "residual scale of the mlp":
        patch("feed_forward", lambda *a: real["feed_forward"](*a) / 0.8)
    elif fault == "final norm":
        w = over(torch.ones_like, "final.norm")
    assert rel(O.forward(cfg, w, ids), good) > 0.1
