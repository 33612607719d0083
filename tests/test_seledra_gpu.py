"""Seledra on the GPU against the plain oracle (seledra_oracle.py): each kernel alone, then the engine in fp32 and
bf16 -- whole prompts, portions, decoding (eager and captured), mixed batches, reused slots and blocks, single keys that
stand out, long decoding, the recurrent state's rules, generation through the scheduler."""
import math

import numpy as np
import pytest
import torch

import seledra_oracle as O
from sinisun_oracle import rotate_half, soft_cap
from test_gefazen import rel, write_model
from test_movalorn_gpu import DT, E, F32_TOL, bf, dev, engine, generate, ids_of, pad, run, stream
from test_seledra import MIXED

pytestmark = pytest.mark.gpu

# (bf16: narrow models; the worst position of hundreds)
TOL = {"float32": F32_TOL, "bfloat16": 7e-2}

# aligned: the decode GEMVs and the prefill GEMMs' own tiles; wide: many query heads per key head, wide states, one tap and
# many; deep: heads above 128 dimensions, the largest states; solo and bare: one kind of layer alone, a factor of 1
ALIGNED = O.make_config(width=512, vocab=640, eps=1e-5, max_positions=600, layers=[
    O.attn_layer(O.dense(768), heads=8, kv_heads=4, dim=64, vdim=64, scale=0.125),
    O.delta_layer(O.dense(512), heads=8, kv_heads=4, dim=64, vdim=64),
    O.delta_layer(O.dense(1024), heads=4, kv_heads=4, dim=128, vdim=128),
    O.attn_layer(O.dense(512), heads=16, kv_heads=4, dim=32, vdim=64, scale=0.2)])
WIDE = O.make_config(width=320, vocab=333, eps=1e-6, residual_mult=1.0, max_positions=512, layers=[
    O.delta_layer(O.dense(72), heads=5, kv_heads=5, dim=150, vdim=72, conv=1),
    O.attn_layer(O.dense(200), heads=34, kv_heads=2, dim=36, vdim=16, scale=0.4),
    O.delta_layer(None, heads=2, kv_heads=1, dim=16, vdim=320, conv=8),
    O.attn_layer(None, heads=2, kv_heads=2, dim=100, vdim=16, scale=0.07)])
DEEP = O.make_config(width=200, vocab=150, residual_mult=1.3, max_positions=512, layers=[
    O.attn_layer(O.dense(33), heads=3, kv_heads=3, dim=144, vdim=200, scale=0.05, v_mix=False),
    O.delta_layer(O.dense(100), heads=3, kv_heads=3, dim=250, vdim=40, conv=3),
    O.attn_layer(None, heads=4, kv_heads=1, dim=256, vdim=250, scale=0.06),
    O.attn_layer(O.dense(10), heads=7, kv_heads=1, dim=13, vdim=250, scale=0.5)])
SOLO = O.make_config(width=512, vocab=130, layers=[
    O.delta_layer(O.dense(4100), heads=3, kv_heads=3, dim=40, vdim=48),
    O.delta_layer(None, heads=4, kv_heads=1, dim=16, vdim=16, conv=6)])
BARE = O.make_config(width=1024, vocab=90, residual_mult=0.5, layers=[
    O.attn_layer(None, heads=2, kv_heads=1, dim=64, vdim=32, scale=0.2),
    O.attn_layer(None, heads=2, kv_heads=1, dim=32, vdim=32, scale=0.2)])
CONFIGS = {"mixed": MIXED, "aligned": ALIGNED, "wide": WIDE, "deep": DEEP, "solo": SOLO, "bare": BARE}
_cache, _want = {}, {}


def model(name, tmp_models, qk_gain=1.5):
    """(folder, config, weights) of a configuration, written once."""
    if name not in _cache:
        cfg = CONFIGS[name]
        w = O.random_weights(cfg, seed=11, qk_gain=qk_gain)
        _cache[name] = (write_model(tmp_models / ("seledra-" + name), cfg, w), cfg, w)
    return _cache[name]


def oracle(name, cfg, w, ids):
    key = (name, tuple(ids))
    if key not in _want:
        _want[key] = O.forward(cfg, w, ids)
    return _want[key]


# ---- kernels alone -----------------------------------------------------------------------------------
DELTA = [(6, 2, 20, 24, 3), (6, 6, 40, 32, 4), (3, 1, 128, 64, 2), (2, 1, 200, 16, 1), (5, 5, 70, 200, 10), (8, 2, 33, 300, 7),
         (1, 1, 64, 640, 4), (4, 2, 180, 72, 4), (32, 16, 128, 128, 4)]


@pytest.mark.parametrize("f32", [0, 1])
@pytest.mark.parametrize("shift", [5, 4])
@pytest.mark.parametrize("sizes", DELTA)
def test_delta_rule_kernels(sizes, shift, f32):
    """Columns at any offset and at aligned ones; portions of unequal lengths at block and chunk borders, continued by others;
    single tokens, some of them twice; slots taken over by a new sequence; state and convolution inputs that no earlier
    sequence may leak; strong and weak decays, and a run of equal keys written at nearly full strength."""
    m = E()
    H, G, N, dv, taps = sizes
    g = torch.Generator().manual_seed(H * 1000 + N)
    rnd = lambda *s: torch.randn(*s, generator=g)
    eps, slots, osc = 3e-4, 6, 0.7
    np_, vp, inner, gn = m.lin_pad_n(N), pad(dv, 16), H * dv, G * N
    dt = torch.float32 if f32 else torch.bfloat16
    norm_w, C = 1 + 0.3 * rnd(dv), inner + 2 * gn
    w = dict(conv_w=rnd(C, taps) / math.sqrt(taps), dt_b=rnd(H) - 2.5, a_log=rnd(H) - 1)
    w["dt_b"][0] = 3.0
    width = 2 * inner + 2 * gn + 2 * H  # [v | k | q | gate | strengths | steps]
    off = dict(x_off=shift, z_off=shift + C, b_off=shift + C + inner, dt_off=shift + C + inner + H, taps=taps, q_scale=N ** -0.5)

    def ref(x, rounded=False):
        x = x.double()
        T = x.shape[0]
        W = {k: v.double() for k, v in w.items()}
        u, z, b, s = torch.split(x, [C, inner, H, H], 1)
        u = O.silu(O.causal_conv(u, W["conv_w"]))
        if rounded:
            u = u.float().bfloat16().double()
        v, k, q = torch.split(u, [inner, gn, gn], 1)
        k, q = (O.unit(y.reshape(T, G, N)).repeat_interleave(H // G, 1) for y in (k, q))
        o = O.delta_rule(O.decay(s, W["a_log"], W["dt_b"]), torch.sigmoid(b), k, v.reshape(T, H, dv), q * N ** -0.5)
        return osc * (O.rms(o, eps) * norm_w.double()).reshape(T, inner) * O.silu(z)

    def inputs(n, steady=False):
        x = rnd(n, width)
        if steady:
            x[20:70, :C] = x[20, :C] + 0.01 * x[20:70, :C]
            x[20:70, C + inner:C + inner + H] += 5
        return bf(x)

    X = {s: inputs(n, s == 1) for s, n in {0: 230, 2: 140, 5: 90, 3: 100, 4: 700, 1: 500}.items()}
    # 16-bit portions round the convolution's outputs: where an output nearly cancels, that is what is left of it
    soft = lambda x: (ref(x, True) - ref(x)).abs().amax(1, keepdim=True) * (0 if f32 else 2)
    want = {s: (ref(x), soft(x)) for s, x in X.items()}
    D = {k: dev(v) for k, v in dict(w, norm_w=norm_w).items()}
    state = torch.full((2, slots, H, np_, vp), 1e30, device="cuda")
    ring = torch.full((slots, taps, C), 1e30, device="cuda")
    nan = float("nan")
    buf = {k: torch.full((2 * 40 * n + 4096,), nan, dtype=torch.float32 if k == "dec" else dt, device="cuda")
           for k, n in zip(("qo", "ko", "kr", "vo", "so", "dec"), m.lin_ws(m.LIN_DELTA, H, G, np_, vp, bool(f32)))}
    work, ld = torch.zeros(64 * 16, dtype=torch.int32, device="cuda"), pad(shift + width + 3, 4) + shift % 4

    def go(entries, decode=False):
        rows = torch.cat([X[s][st:st + n] for s, st, n in entries])
        n = rows.shape[0]
        inp = torch.full((n, ld), 1e30)
        inp[:, shift:shift + width] = rows
        inp, out, y = dev(inp), torch.zeros(n, inner + 64, dtype=dt, device="cuda"), torch.zeros(n, inner, device="cuda")
        pieces, at = [], 0
        for s, st, k in entries:
            pieces.append([at, k, s, st])
            at += k
        pd, sd = (torch.tensor(v, dtype=torch.int32, device="cuda") for v in zip(*[(p[3], p[2]) for p in pieces]))
        print(sizes, shift, f32, entries, flush=True)
        m.lin_scan([] if decode else pieces, kind=m.LIN_DELTA, H=H, G=G, N=N, dv=dv, vp=vp, inp=inp.data_ptr(), ld=ld, **off,
                   **{k: v.data_ptr() for k, v in D.items()}, ring=ring.data_ptr(), state=state.data_ptr(), slots=slots,
                   pos=pd.data_ptr(), slot=sd.data_ptr(), n=n,
                   **{k: v.data_ptr() for k, v in buf.items()}, y=y.data_ptr(), eps=eps, out_scale=osc, out=out.data_ptr(),
                   ldo=inner + 64, f32=f32, work=work.data_ptr(), stream=stream())
        torch.cuda.synchronize()
        exact, slack = (torch.cat([want[s][i][st:st + k] for s, st, k in entries]) for i in (0, 1))
        miss = ((out.cpu()[:, :inner].double() - exact).abs() - slack).clamp(min=0)
        err, mean = float(miss.max() / exact.abs().max()), float(miss.pow(2).mean().sqrt() / exact.pow(2).mean().sqrt())
        print(err, mean, flush=True)
        assert (out[:, inner:] == 0).all() and err < (2e-5 if f32 else 3e-2) and mean < (1e-5 if f32 else 5e-3), (entries, err, mean)

    go([(0, 0, 1), (2, 0, 64), (5, 0, 2), (3, 0, 31)])
    go([(0, 1, 100), (2, 64, 17), (5, 2, 1)])
    go([(0, 101, 1), (5, 3, 1), (3, 31, 1), (2, 81, 1)], True)
    go([(5, 3, 1), (0, 101, 1), (2, 81, 1)], True)                  # once more at the same positions
    go([(5, 4, 1), (2, 82, 1)], True)
    go([(5, 4, 1), (2, 82, 1)])                                     # again, as portions of one token
    go([(2, 83, 48), (0, 102, 128), (3, 32, 66), (5, 5, 3)])        # even lengths: in and out at one parity
    go([(4, 0, 390), (1, 0, 130)])                                  # long, unequal
    go([(1, 130, 370), (4, 390, 1), (5, 8, 2)])                     # from a state, in place (even length)
    go([(4, 391, 309), (5, 10, 6)])
    X[0] = inputs(70)
    want[0] = ref(X[0]), soft(X[0])
    go([(0, 0, 2), (5, 16, 74)])
    go([(0, 2, 1)], True)
    go([(0, 3, 49)])
    X[3] = inputs(9)
    want[3] = ref(X[3]), soft(X[3])
    for t in range(9):
        go([(3, t, 1)], True)


GQA = [(6, 2, 40, 24, 0, 0, 0, 0.0), (9, 3, 14, 28, 0, 0, 0, 0.0), (20, 1, 64, 64, 2, 0, 70, 3.0), (3, 3, 144, 72, 100, 65, 0, 0.0),
       (34, 2, 20, 200, 0, 45, 0, 0.0), (4, 2, 256, 250, 254, 0, 0, 15.0), (32, 8, 128, 128, 0, 0, 0, 0.0), (5, 5, 37, 13, 6, 0, 0, 0.0)]


@pytest.mark.parametrize("f32", [0, 1])
@pytest.mark.parametrize("H, G, dk, dv, rot, window, chunk, cap", GQA)
def test_attention_with_norms_temperatures_and_mixed_values(H, G, dk, dv, rot, window, chunk, cap, f32):
    """Unequal sequences over scattered blocks: single tokens, portions of several through the tiled kernel (key splits)
    and the flash kernel; both layers of a pair whose values are mixed; the norms together with rotation, windows, chunks
    and a cap; every mechanism left out once."""
    m, g = E(), torch.Generator().manual_seed(H * 1000 + dk)
    rnd = lambda *s: torch.randn(*s, generator=g)
    dkp, dvp, maxb, rep = pad(dk, 32), pad(dv, 32), 6, H // G
    lens = [1, 64, 65, 200, 129, 101]
    seqs = [(i, l - 1, 1) for i, l in enumerate(lens)] + [(6, 90, 47)]
    flash = (7, 60, 150)  # (the flash kernel, 16-bit)
    tot = seqs + [flash]
    n, nall, nslot = sum(s[2] for s in seqs), sum(s[2] for s in tot), 8
    scale, osc, base, P, eps = 1.0 / math.sqrt(dk), 0.6, 300.0, maxb * 64, 2e-2
    perm = torch.randperm(nslot * maxb, generator=g).view(nslot, maxb)
    qb, kb, vb, sink = rnd(H * dk), rnd(G * dk), rnd(G * dv), torch.zeros(H)
    qn, kn, temp, lam = 1 + 0.4 * rnd(H * dk), 1 + 0.4 * rnd(G * dk), 1 + 0.4 * rnd(H), torch.tensor([0.35])
    ld, cols = pad(H * dk + G * (dk + dv) + H, 4), H * dk + G * (dk + dv)
    inp, first = rnd(nall, ld), rnd(nall, G, dv)
    ctx = {s: (bf(rnd(st, G, dk)), bf(rnd(st, G, dv))) for s, st, _ in tot}
    turn = lambda v, p: rotate_half(torch.cat([torch.zeros(p, *v.shape[1:], dtype=O.DT), v.double()]), base, rot)[p:]
    blk = torch.zeros(nslot * maxb + 1, G * 64 * (dkp + dvp))
    kview, vview = blk[:, :G * 64 * dkp].view(-1, G, 64, dkp), blk[:, G * 64 * dkp:].view(-1, G, 64, dvp)
    for s, st, _ in tot:
        for p in range(st):
            kview[perm[s, p // 64], :, p % 64, :dk], vview[perm[s, p // 64], :, p % 64, :dv] = ctx[s][0][p], ctx[s][1][p]
    pos, slot, tiles, row = [], [], [], 0
    for s, st, k in tot:
        pos += range(st, st + k)
        slot += [s] * k
        if s != flash[0]:
            tiles += [(f, min(16, (row + k) * rep - f)) for f in range(row * rep, (row + k) * rep, 16)]
        row += k
    r16 = (lambda t: t) if f32 else (lambda t: t.float().bfloat16().double())

    def ref(qk, vn, tm, mix):
        x = inp.double()
        q, k, v = x[:, :H * dk] + qb, x[:, H * dk:(H + G) * dk] + kb, (x[:, (H + G) * dk:cols] + vb).view(nall, G, dv)
        if qk:
            q, k = O.whole_norm(q, qn.double(), eps), O.whole_norm(k, kn.double(), eps)
        v = O.value_norm(v, eps) if vn else v
        mine = v
        v = O.mix_values(v, first.double(), lam.double()) if mix == 2 else v
        gate, want, row = torch.sigmoid(x[:, cols:cols + H]), torch.zeros(nall, H, dv, dtype=O.DT), 0
        for s, st, kk in tot:
            r = slice(row, row + kk)
            Q = turn(q[r].view(kk, H, dk), st)
            K = torch.cat([ctx[s][0].double(), r16(turn(k[r].view(kk, G, dk), st))])
            V = torch.cat([ctx[s][1].double(), r16(v[r])])
            for i in range(kk):
                p = st + i
                a = max(p // chunk * chunk if chunk else 0, p - window + 1 if window else 0)
                for h in range(H):
                    sc = O.scores(Q[i, h], K[a:p + 1, h // rep], scale, temp[h].double() if tm else 1.0)
                    sc = soft_cap(sc, cap) if cap else sc
                    want[row + i, h] = osc * gate[row + i, h] * (O.weights(sc) @ V[a:p + 1, h // rep])
            row += kk
        return want, mine

    ang = torch.arange(P, dtype=O.DT)[:, None] * base ** (-2.0 * torch.arange(rot // 2, dtype=O.DT) / max(rot, 1))
    dt = torch.float32 if f32 else torch.bfloat16
    D = dict(rope=torch.stack([ang.cos(), ang.sin()], -1).float() if rot else torch.zeros(2), sink=sink, qb=qb, kb=kb, vb=vb, inp=inp,
             pos=torch.tensor(pos, dtype=torch.int32), slot=torch.tensor(slot, dtype=torch.int32), bt=perm.int(),
             tiles=torch.tensor(tiles, dtype=torch.int32))
    D = {k: dev(v) for k, v in D.items()}
    part_of = dict(qn=dev(qn), kn=dev(kn), temp=dev(temp), lambda_=dev(lam))
    some = [(0, 0, 1, 0, 64), (1, 0, 0, 0, 1), (0, 1, 0, 2, 3)] if H * dk <= 700 else []
    for qk, vn, tm, mix, nsplit in [(1, 1, 1, 2, 1), (1, 1, 1, 1, 3)] + some:
        want, mine = ref(qk, vn, tm, mix)
        nsplit = 1 if f32 else nsplit
        pool, fd = dev(blk.to(dt)), dev(first if mix == 2 else torch.full_like(first, float("nan")))
        out = torch.zeros(nall, H * dvp, dtype=dt, device="cuda")
        q = torch.zeros(nall, H, dkp, dtype=dt, device="cuda")
        na = nall if f32 else n
        part, ml = torch.zeros(nsplit, na * H, dvp, device="cuda"), torch.zeros(nsplit, na * H, 2, device="cuda")
        kw = {} if f32 else dict(flash_T=flash[2], flash_row0=n, flash_slot=flash[0], flash_start=flash[1])
        use = (["qn", "kn"] if qk else []) + (["temp"] if tm else []) + (["lambda_"] if mix == 2 else [])
        kw.update({k: part_of[k].data_ptr() for k in use}, v_norm=vn, eps=eps, first=fd.data_ptr() if mix else 0)
        print(H, G, dk, dv, rot, window, chunk, cap, f32, qk, vn, tm, mix, nsplit, flush=True)
        m.gqa_attention(rows=nall, n=na, H=H, G=G, dk=dk, dkp=dkp, dv=dv, dvp=dvp, rot=rot, window=window, chunk=chunk, scale=scale,
                        softcap=cap, ld=ld, q_off=0, k_off=H * dk, v_off=(H + G) * dk, g_off=cols, out_scale=osc, pool=pool.data_ptr(),
                        maxb=maxb, f32=f32, q=q.data_ptr(), n_tiles=len(tiles), nsplit=nsplit, opart=part.data_ptr(),
                        ml=ml.data_ptr(), out=out.data_ptr(), ldo=H * dvp, stream=stream(),
                        **{k: v.data_ptr() for k, v in D.items()}, **kw)
        torch.cuda.synchronize()
        got = out.float().cpu().view(nall, H, dvp)
        assert (got[:, :, dv:] == 0).all()
        err = (got[:, :, :dv].double() - want).abs().amax((1, 2)) / want.abs().max()
        assert float(err.max()) < (2e-5 if f32 else 2.5e-2), (nsplit, int(err.argmax()), float(err.max()))
        if mix == 1:
            assert (fd.cpu().double() - mine).abs().max() < 1e-5 * mine.abs().max()


@pytest.mark.parametrize("M", [1, 2, 3, 4, 5, 33, 64, 65, 300])
def test_xielu_in_the_product(M):
    """scale act(W x) in the product's epilogue: GEMV engine, skinny and prefill GEMM, fp32."""
    m, g = E(), torch.Generator().manual_seed(M)
    K, N, p, q, scale = 512, 768, torch.tensor(0.9).double(), torch.tensor(-0.4).double(), 0.6
    x, w = bf(torch.randn(M, K, generator=g)), bf(2 * torch.randn(N, K, generator=g) / math.sqrt(K))
    z = x.double() @ w.double().T
    want = scale * O.xielu(z, p, q)
    qm = m.QMatrix(int(m.QT_BF16), N, K, w.bfloat16().view(torch.int16).numpy())
    xd = dev(x.bfloat16())
    kw = dict(pos=float(O.softplus(p)), neg=float(0.5 + O.softplus(q)), scale=scale)

    def check(y, tol):
        assert (y.cpu().double() - want).abs().max() / want.abs().max() < tol

    y = torch.zeros(M, N, dtype=torch.bfloat16, device="cuda")
    if M <= 4:
        m.gemv([qm], M, 0, K, 0, 1e-5, 0, N, m.EPI_ACT16, stream(), x16=xd.data_ptr(), y16=y.data_ptr(), ldy16=N, act=m.ACT_XIELU, **kw)
        torch.cuda.synchronize()
        check(y, 5e-3)
    y.zero_()
    m.gemm_q(xd.data_ptr(), K, [qm], M, 0, y.data_ptr(), N, m.GEPI_STORE16, stream(), unary=1 + m.ACT_XIELU, **kw)
    torch.cuda.synchronize()
    check(y, 5e-3)
    y32 = torch.zeros(M, N, device="cuda")
    m.bias_act_f32(dev(z.float()).data_ptr(), N, 0, y32.data_ptr(), N, M, N, m.ACT_XIELU, stream(), **kw)
    torch.cuda.synchronize()
    check(y32, 2e-6)


# ---- the engine against the oracle ----------------------------------------------------------------------
@pytest.mark.parametrize("dtype", DT)
@pytest.mark.parametrize("name", list(CONFIGS))
def test_whole_prompt_portions_and_decode(name, dtype, tmp_models):
    path, cfg, w = model(name, tmp_models)
    ids = ids_of(cfg, 270)
    want = oracle(name, cfg, w, ids)
    eng = engine(path, dtype)
    assert rel(run(eng, 0, ids, [len(ids)]), want) < TOL[dtype]
    for slot, sizes in ((1, [2]), (2, [3, 61, 64, 1, 128, 5, 7]), (3, [130, 1]), (1, [1]), (2, [150, 17, 16, 33, 32])):
        n = 40 if sizes in ([2], [1]) else 170
        eng.release_slot(slot)
        assert rel(run(eng, slot, ids[:n], sizes), want[:n]) < TOL[dtype], sizes


@pytest.mark.parametrize("name", ["aligned", "mixed"])
def test_residual_after_every_layer(name, tmp_models):
    path, cfg, w = model(name, tmp_models)
    ids, trace = ids_of(cfg, 50, 9), []
    O.forward(cfg, w, ids, trace)
    eng = engine(path, "float32")
    assert eng.layer_runs == len(trace) == len(cfg["layers"])
    for k in range(len(trace)):
        eng.set_run_limit(k + 1)
        eng.step([0], [0], [50], ids, [])
        assert (torch.from_numpy(eng.last_residual(50)).double() - trace[k]).abs().max() < 1e-4 * max(1.0, float(trace[k].abs().max()))
    eng.set_run_limit(-1)
    assert rel(run(eng, 0, ids, [50]), oracle(name, cfg, w, ids)) < F32_TOL


@pytest.mark.parametrize("name", ["aligned", "wide", "deep"])
def test_long_portions_on_a_long_context(name, tmp_models, monkeypatch):
    """The flash kernel from 32-token portions on, and passes of at most 96 rows: every border between the two
    kernels and between the passes of one step."""
    monkeypatch.setenv("AIOS_GQA_PF_MIN", "32")
    monkeypatch.setenv("AIOS_STEP_ROWS", "96")
    path, cfg, w = model(name, tmp_models)
    ids = ids_of(cfg, 390, 3)
    want = oracle(name, cfg, w, ids)
    eng = engine(path)
    assert rel(run(eng, 0, ids, [390]), want) < TOL["bfloat16"]
    assert rel(run(eng, 1, ids, [33, 31, 64, 2, 100, 97, 32]), want) < TOL["bfloat16"]


@pytest.mark.parametrize("dtype", DT)
@pytest.mark.parametrize("name", ["mixed", "aligned"])
def test_mixed_batches_equal_each_alone(name, dtype, tmp_models):
    """Portions of some requests beside decoded tokens of others; a request pauses; slots and blocks are reused."""
    path, cfg, w = model(name, tmp_models)
    lens = [150, 9, 70, 33, 101, 64]
    seqs = [ids_of(cfg, n, 20 + i) for i, n in enumerate(lens)]
    want = [oracle(name, cfg, w, s) for s in seqs]
    eng = engine(path, dtype, kv_pool_tokens=7 * 64)
    rng = np.random.default_rng(4)
    free, live, todo, got = [0, 1, 2, 3], {}, list(range(6)), [[] for _ in seqs]
    while todo or live:
        while todo and free and sum(-(-lens[i] // 64) for i in list(live) + todo[:1]) <= 7:
            i = todo.pop(0)
            live[i] = [free.pop(), 0]
        entries = [i for i in live if rng.random() < 0.8] or list(live)[:1]
        counts = [min(int(rng.choice([1, 1, 2, 5, 40, 66])), lens[i] - live[i][1]) for i in entries]
        toks = [t for i, n in zip(entries, counts) for t in seqs[i][live[i][1]:live[i][1] + n]]
        out = eng.step([live[i][0] for i in entries], [live[i][1] for i in entries], counts, toks, list(range(len(toks))))
        at = 0
        for i, n in zip(entries, counts):
            got[i].append(torch.from_numpy(out[at:at + n].copy()))
            at += n
            live[i][1] += n
            if live[i][1] == lens[i]:
                eng.release_slot(live[i][0])
                free.append(live.pop(i)[0])
    assert eng.kv_blocks_free == 7
    for i in range(6):
        assert rel(torch.cat(got[i]), want[i]) < TOL[dtype], i


@pytest.mark.parametrize("name", ["mixed", "aligned", "solo", "bare"])
@pytest.mark.parametrize("dtype", DT)
def test_captured_decode_equals_the_oracle(name, dtype, tmp_models):
    """The decode graphs (every batch size's kernels) replayed step after step with other engine work in between, across
    block and chunk borders; logits of every replay."""
    path, cfg, w = model(name, tmp_models)
    seqs = [ids_of(cfg, 60 + 3 * (i % 6), 50 + i % 6) for i in range(40)]
    want = [oracle(name, cfg, w, s) for s in seqs[:6]]
    eng = engine(path, dtype, max_slots=41, max_batch=40, max_ctx=128)
    for B in (1, 2, 4, 5, 6, 40):
        start = [len(s) - 9 for s in seqs[:B]]
        for b in range(B):
            eng.release_slot(b)
            eng.prefill(b, seqs[b][:start[b]], 0, False)
        got = [[] for _ in range(B)]
        for t in range(9):
            eng.decode(list(range(B)), [seqs[b][start[b] + t] for b in range(B)], [start[b] + t for b in range(B)])
            lg = torch.from_numpy(eng.last_logits(B))
            for b in range(B):
                got[b].append(lg[b:b + 1])
            if t == 4:
                eng.prefill(40, seqs[0][:5], 0, True)  # eager work between two replays
        for b in range(B):
            assert rel(torch.cat(got[b]), want[b % 6][start[b]:]) < TOL[dtype], (B, b)


def pair_model(tmp_models):
    """Token 1 asks for token 0: in the attention layers one column of a query and of a key alone stand for the pair, so that
    its score is far above all others; positions and the recurrence stay small."""
    cfg = O.make_config(width=128, vocab=90, eps=1e-5, residual_mult=0.9, max_positions=400, layers=[
        O.attn_layer(O.dense(96), heads=2, kv_heads=1, dim=32, vdim=48, scale=0.3),
        O.delta_layer(None, heads=2, kv_heads=2, dim=8, vdim=16)])
    w = {k: v.float() for k, v in O.random_weights(cfg, 77).items()}
    w["embed"][0, :], w["embed"][1, :] = 0.0, 0.0
    w["embed"][0, 5], w["embed"][1, 9] = 12.0, 12.0
    w["pos"] *= 0.02
    q = "l0.mix."
    for t, col, row in (("q", 9, 20), ("k", 5, 20)):
        w[q + t][:, col], w[q + t + ".b"][:] = 0.0, 0.0
        w[q + t][row, col] = 2.0
    w[q + "g"][0], w[q + "temp"][0] = 0.0, 1.1
    w["l1.mix.o"] *= 0.02
    w = {k: v.to(torch.bfloat16) for k, v in w.items()}
    return write_model(tmp_models / "seledra-pair", cfg, w), cfg, w


@pytest.mark.parametrize("dtype", DT)
def test_single_keys_far_back_and_at_block_borders(dtype, tmp_models, monkeypatch):
    path, cfg, w = pair_model(tmp_models)
    engs = [engine(path, dtype, max_ctx=400)]
    if dtype == "bfloat16":
        monkeypatch.setenv("AIOS_GQA_PF_MIN", "2")  # the flash kernel for every portion
        engs.append(engine(path, dtype, max_ctx=400))
    for n in (2, 17, 64, 65, 66, 129, 193, 300, 400):
        for key in sorted({0, 1, 15, 16, 31, 32, 63, 64, 127, 128, n - 3, n - 2} & set(range(n - 1))):
            ids = [2 + t % 88 for t in ids_of(cfg, n, 300 + n)]
            ids[key], ids[-1] = 0, 1
            want = O.forward(cfg, w, ids)[-1:]
            if n in (129, 300):  # the key is what the last position's logits rest on
                assert rel(O.forward(cfg, w, ids[:key] + [50] + ids[key + 1:])[-1:], want) > 0.15
            for eng in engs:
                for slot, sizes in ((0, [n]), (1, [n - 1, 1]), (2, [40, 29, 2, 100, 1])):
                    eng.release_slot(slot)
                    assert rel(run(eng, slot, ids, sizes)[-1:], want) < 2 * TOL[dtype], (n, key, sizes)


def keep_model(tmp_models):
    """A recurrence that keeps what it is told: no decay to speak of, full strength for token 0, next to none for the others."""
    cfg = O.make_config(width=128, vocab=90, eps=1e-5, residual_mult=1.0, max_positions=600, layers=[
        O.delta_layer(None, heads=4, kv_heads=2, dim=32, vdim=32, conv=3), O.attn_layer(O.dense(64), heads=2, kv_heads=2)])
    w = {k: v.float() for k, v in O.random_weights(cfg, 78).items()}
    w["embed"][:, 7] = -6.0
    w["embed"][0], w["embed"][1] = 0.0, 0.0
    w["embed"][0, 7], w["embed"][1, 7] = 9.0, -9.0
    w["pos"] *= 0.02
    p = "l0.mix."
    w[p + "b"][:], w[p + "b"][:, 7] = 0.0, 2.0
    w[p + "A_log"][:], w[p + "dt_bias"][:] = -4.0, -4.0
    w[p + "a"] *= 0.05
    w["l1.mix.o"] *= 0.05
    w = {k: v.to(torch.bfloat16) for k, v in w.items()}
    return write_model(tmp_models / "seledra-keep", cfg, w), cfg, w


@pytest.mark.parametrize("dtype", DT)
def test_what_the_state_keeps_over_hundreds_of_tokens(dtype, tmp_models):
    path, cfg, w = keep_model(tmp_models)
    eng = engine(path, dtype, max_ctx=600)
    n = 520
    ids = [2 + t % 88 for t in ids_of(cfg, n, 5)]
    ids[3] = 0
    want = O.forward(cfg, w, ids)
    assert rel(O.forward(cfg, w, ids[:3] + [50] + ids[4:])[-1:], want[-1:]) > 0.15
    for slot, sizes in ((0, [n]), (1, [4, 2, 3, 100, 1]), (2, [300, 1, 1, 64])):
        assert rel(run(eng, slot, ids, sizes), want) < TOL[dtype], sizes


@pytest.mark.parametrize("dtype", DT)
def test_the_first_tokens_of_a_sequence(dtype, tmp_models):
    path, cfg, w = model("mixed", tmp_models)
    eng = engine(path, dtype)
    for seed in range(4):
        ids = ids_of(cfg, 5, 700 + seed)
        want = oracle("mixed", cfg, w, ids)
        for slot, sizes in ((0, [5]), (0, [1]), (1, [2, 3]), (1, [1, 4])):  # (slots are taken over without a release)
            assert rel(run(eng, slot, ids, sizes), want) < TOL[dtype]


@pytest.mark.parametrize("dtype", DT)
def test_long_decoding_and_the_context_limit(dtype, tmp_models):
    path, cfg, w = model("mixed", tmp_models)
    P = 300
    ids = ids_of(cfg, P, 8)
    want = oracle("mixed", cfg, w, ids)
    eng = engine(path, dtype, max_ctx=P)
    run(eng, 0, ids[:P - 200], [P - 200])
    assert rel(run(eng, 0, ids[P - 200:], [1], start=P - 200), want[P - 200:]) < TOL[dtype]
    with pytest.raises(RuntimeError, match="overflow"):
        eng.step([0], [P], [1], [0], [])
    with pytest.raises(RuntimeError):
        eng.step([1], [0], [1], [cfg["vocab"]], [])


def test_the_recurrent_state_stands_at_one_position(tmp_models):
    """Where a slot may go on, a dropped single token, copies; anything else is refused before it runs."""
    path, cfg, w = model("mixed", tmp_models)
    a, b = ids_of(cfg, 140, 1), ids_of(cfg, 60, 2)
    eng = engine(path, "float32")
    assert eng.recurrent and eng.resumable(0, 0) and not eng.resumable(0, 1)
    run(eng, 0, a, [140])
    assert eng.resumable(0, 140) and not eng.resumable(0, 139) and not eng.resumable(0, 100)
    for start in (100, 139, 141):
        with pytest.raises(RuntimeError, match="state stands"):
            eng.step([0], [start], [1], [0], [])
    eng.copy_slot(0, 1, 140)
    assert rel(run(eng, 1, b, [60], start=140), O.forward(cfg, w, a + b)[140:]) < F32_TOL
    # a single token whose result is dropped, then another in its place; the copy's state is its own
    run(eng, 0, [5], [1], start=140)
    assert eng.resumable(0, 141) and eng.resumable(0, 140)
    more = ids_of(cfg, 20, 3)
    assert rel(run(eng, 0, more, [1], start=140), O.forward(cfg, w, a + more)[140:]) < F32_TOL


def test_tensor_errors(tmp_models):
    path, cfg, w = model("mixed", tmp_models)
    bad = write_model(tmp_models / "sl-bad", cfg, {k: v for k, v in w.items() if k != "l0.mix.dt_bias"})
    with pytest.raises(ValueError, match="l0.mix.dt_bias"):
        engine(bad)
    bad = write_model(tmp_models / "sl-bad2", cfg, dict(w, **{"l2.mix.q.norm": w["l2.mix.q.norm"][:20]}))
    with pytest.raises(RuntimeError, match="attn_q_norm"):
        engine(bad)
    with pytest.raises(ValueError, match="fp8"):
        engine(path, kv_dtype="fp8")


# ---- generation through the framework's entry points -----------------------------------------------------
@pytest.mark.parametrize("opts", ["#compute=float32", "#compute=float32&kv_tokens=256", ""])
def test_greedy_generation_through_the_scheduler(opts, tmp_models, monkeypatch):
    """Unequal prompts, some of which stop early (the others' queued step is dropped and run again); then a follow-up
    that goes on where the first one's state stands."""
    from aios_amd.runtime.scheduler import GenRequest

    monkeypatch.setenv("AIOS_PREFILL_CHUNK", "48")
    path, cfg, w = model("mixed", tmp_models)
    prompts = [ids_of(cfg, n, 90 + n) for n in (3, 130, 50, 64, 20)]
    n = 12
    key = ("greedy", "mixed")
    if key not in _want:
        _want[key] = [O.greedy(cfg, w, p, n) for p in prompts]
    full = _want[key]
    stop = [full[i][5] if i in (1, 3) else None for i in range(5)]
    reqs = [GenRequest(prompt_ids=p, max_tokens=n, stop_ids=[s] if s is not None else None) for p, s in zip(prompts, stop)]

    def follow(out):
        ids = prompts[0] + out[0][0].token_ids[:-1]
        return [GenRequest(prompt_ids=ids + [7, 8], max_tokens=4)]

    first, second = generate(path + opts, [reqs, follow], 4)
    for p, r, s, f in zip(prompts, first, stop, full):
        if opts:  # 32-bit: the oracle's own choice at every step
            assert r.token_ids == (f if s is None else f[:f.index(s)])
        elif len(r.token_ids):  # bf16: a choice within rounding of the oracle's best, most of the time
            lg = O.forward(cfg, w, p + r.token_ids)[len(p) - 1:-1]
            gap = lg.max(-1).values - lg.gather(1, torch.tensor(r.token_ids)[:, None])[:, 0]
            assert float((gap / lg.std(-1)).median()) < 0.1
    ids = prompts[0] + first[0].token_ids[:-1] + [7, 8]
    if opts:
        assert second[0].token_ids == O.greedy(cfg, w, ids, 4)
    assert len(second[0].token_ids) == 4


def test_synthetic_preset_decodes_and_matches_its_steps():
    """Random-init preset: the captured decode loop's history equals single steps' argmax."""
    from aios_amd.models.config import get_preset
    from aios_amd.runtime.loader import random_engine

    cfg = get_preset("test-seledra")
    eng = random_engine(cfg, seed=3, max_ctx=256, max_slots=2, max_batch=2, compute="float32")
    ids = [int(t) for t in np.random.default_rng(0).integers(0, cfg.vocab_size, 30)]
    first = int(np.asarray(eng.prefill(0, ids, 0, True)).argmax())
    eng.decode_loop_prepare([0], [first], [30])
    eng.decode_loop_run(1, 40, True)
    hist = eng.decode_loop_history(1, 31, 40)
    lg = eng.step([1], [0], [30 + 40], ids + [first] + hist[:39], list(range(29, 70)))
    gap = lg.max(-1) - lg[np.arange(41), [first] + hist]
    assert float((gap / lg.std(-1)).max()) < 1e-3
