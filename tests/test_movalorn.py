"""Movalorn on the CPU: configuration, registry, the scheduler's rules for a recurrent state (fake engine), and the
oracle the GPU tests compare against -- including that each mechanism, left out or shifted by one, would
show in the logits those tests look at."""
import asyncio
import math

import numpy as np
import pytest
import torch

import movalorn_oracle as O
from aios_amd.models import registry
from aios_amd.models.config import LayerConfig, get_preset
from aios_amd.runtime.scheduler import GenRequest, Scheduler
from test_gefazen import MixedEngine, Tok, expected, rel, run_all, write_model

MIXED = O.make_config(loop=(1, 3, 2), layers=[
    O.gru_layer(O.dense(72)), O.attention_layer(O.experts(5, 2, 40, 24)), O.gru_layer(None, width=50),
    O.attention_layer(O.experts(3, 1, 24, None, scale=1.0), heads=5, dim=20, rot_dim=12, vdim=16, kv_rank=72, scale=0.31,
                      window=70, base=500.0)])


def ids_of(n, seed=0, vocab=211):
    return [int(t) for t in np.random.default_rng(seed).integers(0, vocab, n)]


# ---- configuration and checkpoints -----------------------------------------------------------------
def test_config_reads_every_size_and_branch(tmp_path):
    path = write_model(tmp_path / "m", MIXED, O.random_weights(MIXED))
    cfg, raw, arch = registry.load_config(path)
    assert (cfg.vocab_size, cfg.d_model, cfg.norm_eps, cfg.n_layers, cfg.learned_pos) == (211, 96, 3e-5, 4, False)
    assert (cfg.embed_scale, cfg.logit_scale, cfg.bigram, cfg.loop) == (0.8, 0.6, (101, 7, 3), (1, 3, 2))
    common = dict(parallel=False, norm_scalar=True, post_norm=True, resid_gate=True, sink=False)
    assert cfg.layers[0] == LayerConfig(mixer="mingru", width=80, ff=72, act="gelu_tanh", **common)
    assert cfg.layers[1] == LayerConfig(mixer="latent", heads=3, dim=24, vdim=40, kv_rank=56, rot_dim=8, rot_dims=8,
                                        rot_base=3000.0, window=17, scale=0.17, out_gate="head", ff=40, act="silu",
                                        experts=5, top=2, router_scale=1.3, correction=True, shared_ff=24, **common)
    assert cfg.layers[2].ff == 0 and cfg.layers[3].shared_ff == 0 and cfg.layers[3].window == 70
    names = arch.tensor_names(raw)
    assert set(names) == set(O.tensor_shapes(MIXED)) and len(set(names.values())) == len(names)
    assert "l2.norm2" not in names and names["l1.mlp.e4.down"] == "blk.1.ffn_down.4.weight"
    assert registry.is_checkpoint_dir(path)
    assert cfg.n_params() == pytest.approx(sum(math.prod(s) for s in O.tensor_shapes(MIXED).values()), rel=0.02)
    plain = registry.get("movalorn").parse(dict(MIXED, loop=None), "m")
    assert plain.loop is None


@pytest.mark.parametrize("change, message", [
    (dict(type="other"), "mixer type"), (dict(mlp={"kind": "sparse", "ff": 8}), "feed-forward"),
    (dict(mixer=dict(O.attention_layer(None)["mixer"], mask={"size": 0})), "window")])
def test_config_rejects_what_the_design_does_not_have(change, message):
    raw = O.make_config(layers=[dict(O.attention_layer(None), **change)])
    with pytest.raises(ValueError, match=message):
        registry.get("Movalorn").parse(raw, "m")


@pytest.mark.parametrize("loop", [(0, 0, 2), (1, 5, 2), (-1, 2, 2), (0, 1, 0)])
def test_config_rejects_a_loop_that_does_not_fit(loop):
    with pytest.raises(ValueError, match="loop"):
        registry.get("Movalorn").parse(dict(MIXED, loop=dict(zip(("start", "stop", "times"), loop))), "m")


def test_presets_name_the_design():
    for name in ("movalorn-1b", "movalorn-7b", "test-movalorn"):
        cfg = get_preset(name)
        assert cfg.arch == "movalorn" and len(cfg.layers) == cfg.n_layers and cfg.n_params() > 0 and cfg.loop


def test_cpu_backend_refuses_layered_models(tmp_path):
    from aios_amd.runtime.model_manager import ModelManager

    folder = write_model(tmp_path / "m", MIXED, O.random_weights(MIXED))
    m = asyncio.run(ModelManager(max_batch=2, max_slots=2).load_model("movalorn-cpu", folder + "#cpu"))
    assert m.status != "ready" and m.error


# ---- oracle ----------------------------------------------------------------------------------------
def test_oracle_mechanisms_by_hand():
    t = lambda *v: torch.tensor(v, dtype=O.DT)
    assert torch.allclose(O.scalar_norm(t([3.0, -4.0]), torch.tensor(2.0, dtype=O.DT), 0.5), t([3.0, -4.0]) * 2 / math.sqrt(13.0))
    assert O.bigram_rows([4, 5, 6], 10, 3, 7) == [7, (40 + 15) % 7, (50 + 18) % 7]
    v = torch.ones(3, 6, dtype=O.DT)
    r = O.rotate(v, 100.0, 4)
    assert torch.allclose(r[0], v[0]) and torch.allclose(r[:, 4:], v[:, 4:])
    assert torch.allclose(r[2, :2], t(math.cos(2) - math.sin(2), math.cos(2) + math.sin(2)))
    assert torch.allclose(r[2, 2:4], t(math.cos(0.2) - math.sin(0.2), math.cos(0.2) + math.sin(0.2)))
    assert list(O.visible(9, 4)) == [6, 7, 8, 9] and list(O.visible(2, 4)) == [0, 1, 2]
    z, u = t([0.0], [math.log(3.0)]), t([1.5], [-math.log(3.0)])
    s = O.mingru_states(z, u)
    assert torch.allclose(s, t([0.5 * 2.0], [0.25 * 1.0 + 0.75 * 0.25]))
    w = {"router": torch.eye(3, dtype=O.DT), "correction": t(0.0, 5.0, 0.0)}
    pick, wt = O.route(t([2.0, 0.0, 1.0]), w, "", {"top": 2, "scale": 3.0})
    p = torch.softmax(t(2.0, 0.0, 1.0), 0)
    assert pick.tolist() == [[1, 0]] and torch.allclose(wt[0], 3.0 * p[[1, 0]])
    assert O.schedule(MIXED) == [(0, -1), (1, 0), (2, 0), (1, 1), (2, 1), (3, -1)]
    wr = O.random_weights(MIXED, 3)
    ids = ids_of(20)
    assert torch.allclose(O.forward(MIXED, wr, ids)[:9], O.forward(MIXED, wr, ids[:9]))  # causal


FAULTS = ["no gate per head", "no rotation", "rotated by one more", "window one short", "window one long", "no latent norm",
          "no residual gate", "gate after the norm", "no correction", "weights with correction", "renormalised", "silu",
          "no shared expert", "state lost", "candidate", "no bigram", "first token's bigram", "bigram swapped", "no step",
          "loop entered once", "no embedding in the loop", "scale", "shared state"]


@pytest.mark.parametrize("fault", FAULTS)
def test_a_fault_in_any_mechanism_shows(fault, monkeypatch):
    """Planted in the oracle: some logits move by far more than the GPU tests' tolerances (5e-2 in bf16)."""
    cfg, w = MIXED, O.random_weights(MIXED, 1, qk_gain=2.0)
    ids = ids_of(40, 1)
    good = O.forward(cfg, w, ids)
    zero = lambda *ends: {k: (torch.zeros_like(v) if k.endswith(ends) else v) for k, v in w.items()}
    real = {n: getattr(O, n) for n in ("rotate", "latent_attention", "moe", "mingru_states", "sublayer", "visible", "route", "schedule")}
    patch = lambda n, f: monkeypatch.setattr(O, n, f)
    if fault == "no gate per head":
        w = zero("mix.g")
    elif fault == "no rotation":
        patch("rotate", lambda v, b, d: v)
    elif fault == "rotated by one more":
        patch("rotate", lambda v, b, d: real["rotate"](v, b * 3, d))
    elif fault in ("window one short", "window one long"):
        patch("visible", lambda i, n: real["visible"](i, n + (1 if "long" in fault else -1)))
    elif fault == "no latent norm":
        w = {k: (v * 3 if k.endswith("dkv.norm") else v) for k, v in w.items()}
    elif fault == "no residual gate":
        w = zero("rg1", "rg2", "rg1.b", "rg2.b")
    elif fault == "gate after the norm":
        def sub(x, w, p, n, eps, f):
            h = O.scalar_norm(x, w[f"{p}norm{n}"], eps)
            return x + O.scalar_norm(f(h), w[f"{p}norm{n}b"], eps) * torch.sigmoid(h @ w[f"{p}rg{n}"].T + w[f"{p}rg{n}.b"])
        patch("sublayer", sub)
    elif fault == "no correction":
        w = zero("correction")
    elif fault in ("weights with correction", "renormalised"):
        def route(h, w, p, r):
            pick, wt = real["route"](h, w, p, r)
            if fault == "renormalised":
                return pick, wt / wt.sum(-1, keepdim=True)
            return pick, wt + w[p + "correction"][pick]
        patch("route", route)
    elif fault == "silu":
        patch("gelu_tanh", O.silu)
    elif fault == "no shared expert":
        w = zero("shared.down")
    elif fault == "state lost":
        patch("mingru_states", lambda z, u: torch.cat([real["mingru_states"](z[:30], u[:30]), real["mingru_states"](z[30:], u[30:])]))
    elif fault == "candidate":
        patch("mingru_states", lambda z, u: real["mingru_states"](z, torch.where(u >= 0, u, u - 9)))
    elif fault == "no bigram":
        w = zero("bigram")
    elif fault == "first token's bigram":
        patch("bigram_rows", lambda t, a, b, n: [(t[i - 1] * a + t[i] * b) % n if i else t[0] * b % n for i in range(len(t))])
    elif fault == "bigram swapped":
        cfg = dict(cfg, embedding=dict(cfg["embedding"], bigram={"buckets": 101, "mul_prev": 3, "mul_cur": 7}))
    elif fault == "no step":
        w = zero("loop.step")
    elif fault == "loop entered once":
        patch("schedule", lambda c: [(i, t if t <= 0 or i != 1 else -1) for i, t in real["schedule"](c)])
    elif fault == "no embedding in the loop":
        w = dict(w, **{"loop.in": torch.cat([w["loop.in"][:, :96], torch.zeros(96, 96).bfloat16()], 1)})
    elif fault == "scale":
        cfg = dict(cfg, layers=[dict(l, mixer=dict(l["mixer"], scale=0.125)) for l in cfg["layers"]])
    elif fault == "shared state":
        seen = []
        def states(z, u):
            s = real["mingru_states"](z, u, seen[-1] if len(seen) == 2 else None)
            seen.append(s[-1])
            return s
        patch("mingru_states", states)
    assert rel(O.forward(cfg, w, ids), good) > 0.1


# ---- scheduler: recurrent state ---------------------------------------------------------------------------
class RecurrentEngine(MixedEngine):
    """MixedEngine whose slots hold a state at one position, with the last single token repeatable."""
    recurrent = True

    def __init__(self, slots, blocks):
        super().__init__(slots, blocks)
        self.at = {s: (0, False) for s in range(slots)}
        self.copies, self.pend = [], None

    def resumable(self, s, n):
        pos, again = self.at[s]
        return n == 0 or n == pos or (again and n == pos - 1)

    def _move(self, s, start, n):
        assert self.resumable(s, start), (s, start, self.at[s])
        self.at[s] = (start + n, n == 1)

    def release_slot(self, s):
        super().release_slot(s)
        self.at[s] = (0, False)

    def copy_slot(self, src, dst, n):
        assert self.resumable(src, n)
        self.copies.append((src, dst, n))
        self.at[dst] = self.at[src]

    def prefill(self, slot, ids, start, want=True):
        self._move(slot, start, len(ids))
        return super().prefill(slot, ids, start, want)

    def step_sample(self, slots, starts, counts, *a):
        for s, st, n in zip(slots, starts, counts):
            self._move(s, st, n)
        return super().step_sample(slots, starts, counts, *a)

    # pipelined decode: the forward moves the state at once, the token follows
    def decode_submit(self, slots, toks, pos, *a):
        if toks:
            self.last = list(toks)
        for s, p in zip(slots, pos):
            self._move(s, p, 1)
            self._write(s, p + 1)
        self.pend = list(zip(pos, range(len(slots))))

    def decode_sample(self, mask):
        self.out = [self.nxt(self.last[i], p) for p, i in self.pend]
        self.last = self.out

    def decode_collect(self):
        return self.out


def test_scheduler_keeps_a_recurrent_state_in_step():
    """Requests of unequal lengths: whenever one ends, the queued step of the others is dropped and run again."""
    eng = RecurrentEngine(4, 4 * 64)
    sched = Scheduler(eng, Tok(), max_batch=4, max_slots=4, max_ctx=256)
    try:
        prompts = [[i + 3] * n for i, n in enumerate((5, 40, 11, 23, 9, 17))]
        reqs = []
        for i, p in enumerate(prompts):
            stop = [expected(p, 30)[6 + 3 * i]]  # ends at a token nobody knows in advance
            reqs.append(GenRequest(prompt_ids=p, max_tokens=30, stop_ids=stop))
        res = run_all(sched, reqs)
    finally:
        sched.close()
    for i, (p, r) in enumerate(zip(prompts, res)):
        want = expected(p, 30)
        assert r.finish_reason == "stop" and r.token_ids == want[:want.index(want[6 + 3 * i])], r


def test_scheduler_reuses_a_prefix_only_where_the_state_stands():
    eng = RecurrentEngine(3, 3 * 256)
    sched = Scheduler(eng, Tok(), max_batch=3, max_slots=3, max_ctx=1024)
    try:
        first = [5] * 200
        r = run_all(sched, [GenRequest(prompt_ids=first, max_tokens=8)])[0]
        taken_in = first + r.token_ids[:-1]  # (the last sampled token was never fed)
        follow = taken_in + [9] * 30
        r2 = run_all(sched, [GenRequest(prompt_ids=follow, max_tokens=8)])[0]
        assert r2.cached_prompt_tokens == len(taken_in) and r2.token_ids == expected(follow, 8)
        half = first[:150] + [8] * 20         # a prefix the state has gone past
        r3 = run_all(sched, [GenRequest(prompt_ids=half, max_tokens=8)])[0]
        assert r3.cached_prompt_tokens == 0 and r3.token_ids == expected(half, 8) and not eng.copies
    finally:
        sched.close()
