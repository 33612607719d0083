"""Gefazen on the GPU against the plain oracle (gefazen_oracle.py): each kernel alone, then the engine in fp32
and bf16 -- whole prompts, portions, decoding (eager and captured), mixed batches, reused slots and blocks, keys at
block borders, long decoding, generation through the scheduler."""
import math
import threading

import numpy as np
import pytest
import torch

import gefazen_oracle as O
from test_gefazen import MIXED, rel, write_model

pytestmark = pytest.mark.gpu

F32_TOL, BF16_TOL = 2e-5, 3e-2
TOL = {"float32": F32_TOL, "bfloat16": BF16_TOL}
DT = list(TOL)

# the aligned shape takes the decode GEMVs and the prefill GEMMs' own tiles; wide: more than 16 heads, a rank
# with an odd number of 64-column tiles; deep: rank above 256, head dimensions above 64 and unequal
ALIGNED = O.make_config(width=512, vocab=640, max_positions=700, eps=1e-5, layers=[
    O.make_layer(heads=4, dim=64, vdim=64, kv_rank=128, scale=0.11, ff=768),
    O.make_layer(heads=8, dim=32, vdim=64, kv_rank=64, scale=0.2, ff=None),
    O.make_layer(heads=4, dim=64, vdim=64, kv_rank=128, scale=0.11, ff=768, weights_of=0)])
WIDE = O.make_config(width=320, vocab=333, max_positions=400, eps=1e-6, layers=[
    O.make_layer(heads=20, dim=32, vdim=16, kv_rank=160, scale=0.15, ff=200),
    O.make_layer(heads=1, dim=96, vdim=160, kv_rank=40, scale=0.09, ff=64)])
DEEP = O.make_config(width=200, vocab=150, max_positions=300, layers=[
    O.make_layer(heads=3, dim=144, vdim=72, kv_rank=300, scale=0.08, ff=100),
    O.make_layer(heads=2, dim=20, vdim=200, kv_rank=520, scale=0.25, ff=None)])
CONFIGS = {"mixed": MIXED, "aligned": ALIGNED, "wide": WIDE, "deep": DEEP}
_cache = {}


def model(name, tmp_models, qk_gain=2.0):
    """(folder, config, weights) of a configuration, written once."""
    if name not in _cache:
        cfg = CONFIGS[name]
        w = O.random_weights(cfg, seed=len(_cache) + 11, qk_gain=qk_gain)
        _cache[name] = (write_model(tmp_models / name, cfg, w), cfg, w)
    return _cache[name]


def engine(path, dtype="bfloat16", **kw):
    from aios_amd.runtime.loader import load_engine

    kw = dict(dict(max_slots=4, max_batch=8), **kw)
    return load_engine(path, compute=dtype, **kw)[0]


def ids_of(cfg, n, seed=0):
    return [int(t) for t in np.random.default_rng(seed).integers(0, cfg["vocab"], n)]


def run(eng, slot, ids, sizes, start=0):
    """Feed ids in portions of the given sizes (the last repeats); logits of every position."""
    out, at, k = [], 0, 0
    while at < len(ids):
        n = min(sizes[min(k, len(sizes) - 1)], len(ids) - at)
        out.append(eng.step([slot], [start + at], [n], ids[at:at + n], list(range(n))))
        at += n
        k += 1
    return torch.from_numpy(np.concatenate(out))


# ---- kernels alone -----------------------------------------------------------------------------------
def dev(t):
    return t.cuda().contiguous()


def E():
    from aios_amd.runtime import native

    return native.require()


def stream():
    return torch.cuda.current_stream().cuda_stream


def pad(n, m):
    return (n + m - 1) // m * m


@pytest.mark.parametrize("f32", [0, 1])
@pytest.mark.parametrize("H, dk, dv, rank, sink, gate", [
    (4, 64, 64, 96, 1, 1), (20, 24, 40, 150, 1, 0), (1, 128, 128, 512, 0, 1), (33, 48, 16, 700, 1, 1), (2, 32, 32, 1000, 1, 1)])
def test_latent_attention_kernel(H, dk, dv, rank, sink, gate, f32):
    """Absorbed attention over a paged cache whose blocks are scattered: unequal sequences (one token each, as
    in decoding, and a portion of several), several key splits, lengths at block borders."""
    g = torch.Generator().manual_seed(H * 1000 + rank)
    rnd = lambda *s: torch.randn(*s, generator=g)
    dkp, dvp = pad(dk, 32), pad(dv, 32)
    rp = next(64 * t for t in (2, 4, 6, 8, 12, 16, 32) if rank <= 64 * t)
    lens, portion, kvb, maxb = [1, 64, 65, 200], 7, 64, 6
    seqs = [(i, l - 1, 1) for i, l in enumerate(lens)] + [(4, 122, portion)]  # slot, start, new tokens
    n = sum(s[2] for s in seqs)
    bf = lambda t: t.to(torch.bfloat16).float()
    uk, uv = bf(rnd(H, dk, rank) / math.sqrt(rank)), bf(rnd(H, dv, rank) / math.sqrt(rank))
    kvn, snk = 1 + 0.2 * rnd(rank), rnd(H) * 2
    scale, eps = 0.6 / math.sqrt(dk) * 3, 1e-5
    perm = torch.randperm(5 * maxb, generator=g).view(5, maxb)
    pool = torch.zeros(5 * maxb + 1, kvb, rp)
    ctx = {s: bf(rnd(start, rank)) for s, start, _ in seqs}
    for s, start, _ in seqs:
        for p in range(start):
            pool[perm[s, p // kvb], p % kvb, :rank] = ctx[s][p]
    dkv_off, g_off, ld = pad(H * dkp, 64), pad(H * dkp, 64) + rp, pad(H * dkp, 64) + rp + pad(H * dvp, 64)
    qdg = torch.zeros(n, ld)
    q, dkv, gt = rnd(n, H, dk) * 2, rnd(n, rank), rnd(n, H, dv)
    qdg[:, :H * dkp].view(n, H, dkp)[:, :, :dk] = q
    qdg[:, dkv_off:dkv_off + rank] = dkv
    qdg[:, g_off:g_off + H * dvp].view(n, H, dvp)[:, :, :dv] = gt
    pos, slot, tiles, row = [], [], [], 0
    for s, start, k in seqs:
        pos += list(range(start, start + k))
        slot += [s] * k
        tiles += [(f, min(16, (row + k) * H - f)) for f in range(row * H, (row + k) * H, 16)]
        row += k
    # expected
    c_new = O.rms_norm(dkv.double(), kvn.double(), eps)
    if not f32:
        c_new = c_new.to(torch.bfloat16).double()
    want, row = torch.zeros(n, H, dv, dtype=O.DT), 0
    for s, start, k in seqs:
        c = torch.cat([ctx[s].double(), c_new[row:row + k]])
        for i in range(k):
            cc = c[:start + i + 1]
            for h in range(H):
                a = (cc @ uk[h].double().T) @ q[row + i, h].double() * scale
                p = O.sink_softmax(a, float(snk[h]) if sink else -1e9)
                o = p @ (cc @ uv[h].double().T)
                want[row + i, h] = o * torch.sigmoid(gt[row + i, h].double()) if gate else o
        row += k
    dt = torch.float32 if f32 else torch.bfloat16
    wukT = torch.zeros(H, rp, dkp)
    wukT[:, :rank, :dk] = uk.transpose(1, 2)
    wuv = torch.zeros(H, dvp, rp)
    wuv[:, :dv, :rank] = uv
    D = dict(norm=torch.zeros(rp), pool=pool.to(dt), wukT=wukT.bfloat16(), wuv=wuv.bfloat16(), qdg=qdg, sink=snk,
             bt=perm.int(), pos=torch.tensor(pos, dtype=torch.int32), slot=torch.tensor(slot, dtype=torch.int32),
             tiles=torch.tensor(tiles, dtype=torch.int32))
    D["norm"][:rank] = kvn
    D = {k: dev(v) for k, v in D.items()}
    for nsplit in (1,) if f32 else (1, 3, 64):
        out = torch.zeros(n, H * dvp, dtype=dt, device="cuda")
        qa = torch.zeros(n, H, rp, dtype=dt, device="cuda")
        part = torch.zeros(nsplit, n * H, rp, device="cuda")
        ml = torch.zeros(nsplit, n * H, 2, device="cuda")
        E().latent_attention(n, n, H, dk, dkp, dvp, rank, rp, scale, eps, D["norm"].data_ptr(),
                             D["sink"].data_ptr() if sink else 0, D["qdg"].data_ptr(), ld, dkv_off, g_off if gate else -1,
                             D["pos"].data_ptr(), D["slot"].data_ptr(), D["pool"].data_ptr(), D["bt"].data_ptr(), maxb, kvb,
                             f32, D["wukT"].data_ptr(), D["wuv"].data_ptr(), qa.data_ptr(), D["tiles"].data_ptr(), len(tiles),
                             nsplit, part.data_ptr(), ml.data_ptr(), out.data_ptr(), H * dvp, stream())
        torch.cuda.synchronize()
        got = out.float().cpu().view(n, H, dvp)
        assert (got[:, :, dv:] == 0).all()
        err = (got[:, :, :dv].double() - want).abs().max() / want.abs().max()
        assert err < (2e-5 if f32 else 2e-2), (nsplit, float(err))


@pytest.mark.parametrize("H, dk, dv, start, T, sink, gate", [
    (2, 64, 64, 0, 300, 1, 1), (3, 24, 40, 77, 2, 1, 1), (1, 128, 128, 63, 130, 0, 0), (2, 160, 96, 128, 65, 1, 0),
    (2, 200, 256, 0, 129, 1, 1), (4, 128, 64, 190, 64, 0, 1)])
def test_mha_prefill_kernel(H, dk, dv, start, T, sink, gate):
    g = torch.Generator().manual_seed(T * 7 + dk)
    rnd = lambda *s: torch.randn(*s, generator=g)
    dkp, dvp, S = pad(dk, 32), pad(dv, 32), start + T
    q, k, v, gt = rnd(T, H, dk), rnd(S, H, dk).bfloat16(), rnd(S, H, dv).bfloat16(), rnd(T, H, dv)
    snk, scale = rnd(H) * 3, 3 / math.sqrt(dk)
    want = torch.zeros(T, H, dv, dtype=O.DT)
    for i in range(T):
        for h in range(H):
            n = start + i + 1
            p = O.sink_softmax((k[:n, h].double() @ q[i, h].double()) * scale, float(snk[h]) if sink else -1e9)
            want[i, h] = p @ v[:n, h].double() * (torch.sigmoid(gt[i, h].double()) if gate else 1.0)
    ldq = H * (dkp + dvp)
    qb = torch.zeros(T, ldq)
    qb[:, :H * dkp].view(T, H, dkp)[:, :, :dk] = q
    qb[:, H * dkp:].view(T, H, dvp)[:, :, :dv] = gt
    kv = torch.zeros(S, ldq, dtype=torch.bfloat16)
    kv[:, :H * dkp].view(S, H, dkp)[:, :, :dk] = k
    kv[:, H * dkp:].view(S, H, dvp)[:, :, :dv] = v
    qb, kv, snk = dev(qb), dev(kv), dev(snk)
    out = torch.zeros(T, H * dvp, dtype=torch.bfloat16, device="cuda")
    E().mha_prefill(qb.data_ptr(), ldq, kv.data_ptr(), kv.data_ptr() + 2 * H * dkp, ldq, H, dkp, dvp, start, T, scale,
                    snk.data_ptr() if sink else 0, qb.data_ptr() + 4 * H * dkp if gate else 0, out.data_ptr(), H * dvp,
                    stream())
    torch.cuda.synchronize()
    got = out.float().cpu().view(T, H, dvp)[:, :, :dv].double()
    err = (got - want).abs().max() / want.abs().max()
    assert err < 2e-2, float(err)


@pytest.mark.parametrize("M, N, K", [(1, 64, 64), (3, 130, 192), (70, 200, 1024), (65, 64, 16)])
def test_gemm_f32_is_32_bit(M, N, K):
    A, W, C = torch.randn(M, K), torch.randn(N, K).bfloat16(), torch.randn(M, N)
    a, w, c = dev(A), dev(W), dev(C)
    E().gemm_f32(a.data_ptr(), K, w.data_ptr(), K, M, N, K, c.data_ptr(), N, 1, stream())
    torch.cuda.synchronize()
    want = C.double() + A.double() @ W.double().T
    assert (c.cpu().double() - want).abs().max() < 3e-6 * math.sqrt(K) * 4


def test_embedding_and_glu_kernels():
    V, P, d, n = 50, 40, 192, 9
    tab, pt = torch.randn(V, d).bfloat16(), torch.randn(P, d).bfloat16()
    tok, pos = torch.randint(0, V, (n,), dtype=torch.int32), torch.randint(0, P, (n,), dtype=torch.int32)
    D = [dev(t) for t in (tab, pt, tok, pos)]
    x = torch.zeros(n, d, device="cuda")
    for use in (1, 0):
        E().embed_pos(D[0].data_ptr(), D[1].data_ptr() if use else 0, D[2].data_ptr(), D[3].data_ptr(), n, d, x.data_ptr(), stream())
        torch.cuda.synchronize()
        assert torch.equal(x.cpu(), tab.float()[tok.long()] + (pt.float()[pos.long()] if use else 0))
    z = torch.randn(3, 2 * 70) * 4
    zd, o = dev(z), torch.zeros(3, 70, device="cuda")
    for act, f in ((1, O.gelu_tanh), (0, torch.nn.functional.silu)):
        E().glu_f32(zd.data_ptr(), 140, o.data_ptr(), 70, 3, 70, act, stream())
        torch.cuda.synchronize()
        assert (o.cpu().double() - f(z[:, ::2].double()) * z[:, 1::2].double()).abs().max() < 1e-5


@pytest.mark.parametrize("M", [1, 3, 4, 9, 40, 64, 100, 300])
def test_fused_projection_epilogues(M):
    """One matrix holding plain rows and interleaved gate / up rows, its epilogues in every product that serves it
    (decode GEMV with the norm in front, skinny GEMM, prefill GEMM), both activations; the bf16 store."""
    m = E()
    K, N0, F = 512, 192, 256
    W = (torch.randn(N0 + 2 * F, K) / math.sqrt(K)).bfloat16()
    x, nw = torch.randn(M, K), 1 + 0.1 * torch.randn(K)
    q = m.QMatrix(int(m.QT_BF16), N0 + 2 * F, K, W.view(torch.int16).numpy())
    q0 = m.QMatrix(int(m.QT_BF16), N0, K, W[:N0].contiguous().view(torch.int16).numpy())
    q1 = m.QMatrix(int(m.QT_BF16), 2 * F, K, W[N0:].contiguous().view(torch.int16).numpy())
    h = O.rms_norm(x.double(), nw.double(), 1e-5)
    y = h @ W.double().T
    for act, f in ((1, O.gelu_tanh), (0, torch.nn.functional.silu)):
        glu = f(y[:, N0::2]) * y[:, N0 + 1::2]
        C = torch.zeros(M, N0, device="cuda")
        G = torch.zeros(M, F + 64, dtype=torch.bfloat16, device="cuda")  # (a wider buffer: the GLU at column 64)
        xd, nd, hd = dev(x), dev(nw), dev(h.bfloat16())
        g64 = G.data_ptr() + 128
        if M <= 4:
            m.gemv([q], M, xd.data_ptr(), K, nd.data_ptr(), 1e-5, C.data_ptr(), N0, m.EPI_STORE_GLU, stream(), y16=g64,
                   act=act, glu_row0=N0, ldy16=F + 64)
        elif M <= 64:
            m.gemm_q(hd.data_ptr(), K, [q], M, C.data_ptr(), g64, N0, m.GEPI_STORE_GLU, stream(), act=act, glu_n0=N0,
                     ldc16=F + 64)
        else:
            m.gemm_q(hd.data_ptr(), K, [q0], M, C.data_ptr(), 0, N0, m.GEPI_STORE, stream())
            m.gemm_q(hd.data_ptr(), K, [q1], M, 0, g64, F + 64, m.GEPI_SWIGLU_BF16, stream(), act=act)
        torch.cuda.synchronize()
        assert (C.cpu().double() - y[:, :N0]).abs().max() < 3e-2
        assert (G.cpu().double()[:, 64:] - glu).abs().max() < 6e-2 and (G[:, :64] == 0).all()
    S = torch.zeros(M, N0, dtype=torch.bfloat16, device="cuda")
    m.gemm_q(hd.data_ptr(), K, [q0], M, 0, S.data_ptr(), N0, m.GEPI_STORE16, stream())
    torch.cuda.synchronize()
    assert (S.cpu().double() - y[:, :N0]).abs().max() < 4e-2


# ---- the engine against the oracle ----------------------------------------------------------------------
@pytest.mark.parametrize("dtype", DT)
@pytest.mark.parametrize("name", list(CONFIGS))
def test_whole_prompt_portions_and_decode(name, dtype, tmp_models):
    path, cfg, w = model(name, tmp_models)
    ids = ids_of(cfg, 270)
    want = O.forward(cfg, w, ids)
    eng = engine(path, dtype)
    tol = TOL[dtype]
    whole = run(eng, 0, ids, [len(ids)])
    assert rel(whole, want) < tol
    for slot, sizes in ((1, [2]), (2, [3, 61, 64, 1, 128, 5, 7]), (3, [130, 1]), (1, [1])):
        n = 40 if sizes in ([2], [1]) else 160
        eng.release_slot(slot)
        got = run(eng, slot, ids[:n], sizes)
        assert rel(got, want[:n]) < tol, (sizes, rel(got, want[:n]))


@pytest.mark.parametrize("name", ["aligned", "wide"])
def test_long_portions_on_a_long_context(name, tmp_models, monkeypatch):
    """Expanded attention from 32-token portions on, and passes of at most 96 rows: every border between the two
    forms and between the passes of one step."""
    monkeypatch.setenv("AIOS_LATENT_PF_MIN", "32")
    monkeypatch.setenv("AIOS_STEP_ROWS", "96")
    path, cfg, w = model(name, tmp_models)
    ids = ids_of(cfg, 390, 3)
    want = O.forward(cfg, w, ids)
    eng = engine(path)
    assert rel(run(eng, 0, ids, [390]), want) < BF16_TOL
    assert rel(run(eng, 1, ids, [33, 31, 64, 2, 100, 97, 32]), want) < BF16_TOL


@pytest.mark.parametrize("dtype", DT)
@pytest.mark.parametrize("name", ["mixed", "aligned"])
def test_mixed_batches_equal_each_alone(name, dtype, tmp_models):
    """Portions of some requests beside decoded tokens of others; a request pauses; slots and blocks are reused."""
    path, cfg, w = model(name, tmp_models)
    lens = [150, 9, 70, 33, 101, 64]
    seqs = [ids_of(cfg, n, 20 + i) for i, n in enumerate(lens)]
    want = [O.forward(cfg, w, s) for s in seqs]
    # the pool holds the four live requests at most: 3 + 1 + 2 + 1 blocks and little more
    eng = engine(path, dtype, kv_pool_tokens=7 * 64)
    assert eng.kv_blocks_total == 7 and eng.kv_block_tokens == 64
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
    with pytest.raises(RuntimeError, match="pool exhausted"):
        eng.step([0], [0], [8 * 64 - 1], ids_of(cfg, 8 * 64 - 1), [])


@pytest.mark.parametrize("name", ["mixed", "aligned"])
@pytest.mark.parametrize("dtype", DT)
def test_captured_decode_equals_the_oracle(name, dtype, tmp_models):
    """The decode graphs (every batch size's kernels: GEMV, skinny GEMM) replayed step after step with other engine
    work in between, across a block border; logits of every replay."""
    path, cfg, w = model(name, tmp_models)
    seqs = [ids_of(cfg, 60 + 3 * i, 50 + i) for i in range(6)]
    want = [O.forward(cfg, w, s) for s in seqs]
    eng = engine(path, dtype, max_slots=8, max_batch=8)
    for B in (1, 2, 4, 5, 6):
        start = [len(s) - 9 for s in seqs[:B]]
        for b in range(B):
            eng.release_slot(b)
            eng.prefill(b, seqs[b][:start[b]], 0, False)
        for t in range(9):
            eng.decode(list(range(B)), [seqs[b][start[b] + t] for b in range(B)], [start[b] + t for b in range(B)])
            lg = torch.from_numpy(eng.last_logits(B))
            for b in range(B):
                assert rel(lg[b:b + 1], want[b][start[b] + t:start[b] + t + 1]) < TOL[dtype], (B, t, b)
            if t == 4:
                eng.prefill(7, seqs[0][:5], 0, True)  # eager work between two replays


def far_model(tmp_models):
    """Token 1 asks for token 0: the first layer's head 0 gives that pair a score far above all others."""
    cfg = O.make_config(width=128, vocab=90, max_positions=600, eps=1e-5, layers=[
        O.make_layer(heads=2, dim=32, vdim=48, kv_rank=64, scale=0.3, ff=96), O.make_layer(heads=3, dim=16, vdim=16, kv_rank=24, ff=None)])
    w = {k: v.float() for k, v in O.random_weights(cfg, 77).items()}
    w["embed"][0, :], w["embed"][1, :] = 0.0, 0.0
    w["embed"][0, 5], w["embed"][1, 9] = 12.0, 12.0
    w["pos"] *= 0.2
    w["l0.mix.dkv"][:, 5] = 0
    w["l0.mix.dkv"][3, 5] = 3.0
    w["l0.mix.uk"][7, 3] = 2.0
    w["l0.mix.q"][7, 9] = 2.0
    w["l0.mix.uv"][:48, 3] *= 3
    w = {k: v.to(torch.bfloat16) for k, v in w.items()}
    return write_model(tmp_models / "far", cfg, w), cfg, w


@pytest.mark.parametrize("dtype", DT)
def test_far_keys_at_block_borders(dtype, tmp_models):
    path, cfg, w = far_model(tmp_models)
    eng = engine(path, dtype)
    n = 330
    for i, p in enumerate((0, 1, 62, 63, 64, 65, 127, 128, 191, 192, 255, 256, 319, 320, n - 2)):
        ids = [2 + t % 88 for t in ids_of(cfg, n, 300 + i)]
        ids[p], ids[-1] = 0, 1
        want = O.forward(cfg, w, ids)[-1:]
        without = O.forward(cfg, w, ids[:p] + [50] + ids[p + 1:])[-1:]
        assert rel(without, want) > 0.15  # the key is what the last position's logits rest on
        for slot, sizes in ((0, [n]), (1, [n - 1, 1]), (2, [100, 64, 2, 163, 1])):
            eng.release_slot(slot)
            assert rel(run(eng, slot, ids, sizes)[-1:], want) < 2 * TOL[dtype], (p, sizes)


@pytest.mark.parametrize("dtype", DT)
def test_long_decoding_and_the_position_limit(dtype, tmp_models):
    path, cfg, w = model("mixed", tmp_models)
    P = cfg["max_positions"]
    ids = ids_of(cfg, P, 8)
    want = O.forward(cfg, w, ids)
    eng = engine(path, dtype)
    run(eng, 0, ids[:P - 200], [P - 200])
    got = run(eng, 0, ids[P - 200:], [1], start=P - 200)
    assert rel(got, want[P - 200:]) < TOL[dtype]
    with pytest.raises(RuntimeError, match="overflow"):
        eng.step([0], [P], [1], [0], [])
    with pytest.raises(RuntimeError):
        eng.step([1], [0], [1], [cfg["vocab"]], [])


def test_prefix_sharing_copies_the_latent_cache(tmp_models):
    path, cfg, w = model("mixed", tmp_models)
    a, b = ids_of(cfg, 140, 1), ids_of(cfg, 60, 2)
    eng = engine(path, "float32")
    run(eng, 0, a, [140])
    eng.copy_slot(0, 1, 100)
    ids = a[:100] + b
    got = run(eng, 1, b, [60], start=100)
    assert rel(got, O.forward(cfg, w, ids)[100:]) < F32_TOL
    more = ids_of(cfg, 20, 3)
    got = run(eng, 0, more, [1], start=140)  # the source's own blocks are untouched
    assert rel(got, O.forward(cfg, w, a + more)[140:]) < F32_TOL


def test_tensor_errors(tmp_models):
    path, cfg, w = model("mixed", tmp_models)
    bad = write_model(tmp_models / "bad", cfg, {k: v for k, v in w.items() if k != "l1.mix.g"})
    with pytest.raises(ValueError, match="l1.mix.g"):
        engine(bad)
    bad = write_model(tmp_models / "bad2", cfg, dict(w, **{"l1.mix.g": w["l1.mix.g"][:3]}))
    with pytest.raises(RuntimeError, match="attn_gate"):
        engine(bad)
    with pytest.raises(ValueError, match="fp8"):
        engine(path, kv_dtype="fp8")


# ---- generation through the framework's entry points -----------------------------------------------------
def generate(mgr_path, prompts, n, max_batch, env=None):
    """Greedy token ids of several prompts submitted at once, through ModelManager and its Scheduler."""
    import asyncio

    from aios_amd.runtime.model_manager import ModelManager
    from aios_amd.runtime.scheduler import GenRequest

    mgr = ModelManager(max_batch=max_batch, max_slots=max_batch)
    m = asyncio.run(mgr.load_model("gefazen-test", mgr_path))
    assert m.status == "ready", m.error
    try:
        res, ev = {}, threading.Event()

        def done(i):
            def f(r):
                res[i] = r
                if len(res) == len(prompts):
                    ev.set()
            return f

        reqs = [GenRequest(prompt_ids=p, max_tokens=n, on_done=done(i)) for i, p in enumerate(prompts)]
        with m.scheduler.cv:
            m.scheduler.queue.extend(reqs)
            m.scheduler.cv.notify()
        assert ev.wait(100)
        return [res[i] for i in range(len(prompts))]
    finally:
        asyncio.run(mgr.unload_model("gefazen-test"))


@pytest.mark.parametrize("opts", ["#compute=float32", "#compute=float32&kv_tokens=256", ""])
def test_greedy_generation_through_the_scheduler(opts, tmp_models, monkeypatch):
    monkeypatch.setenv("AIOS_PREFILL_CHUNK", "48")
    path, cfg, w = model("mixed", tmp_models)
    prompts = [ids_of(cfg, n, 90 + n) for n in (3, 130, 50, 64, 20)]
    n = 12
    res = generate(path + opts, prompts, n, 4)
    for p, r in zip(prompts, res):
        assert r.finish_reason == "length" and len(r.token_ids) == n, r
        lg = O.forward(cfg, w, p + r.token_ids)[len(p) - 1:-1]
        if opts:  # 32-bit: the oracle's own choice at every step
            assert r.token_ids == [int(t) for t in lg.argmax(-1)]
        else:     # bf16: a choice within rounding of the oracle's best
            gap = lg.max(-1).values - lg.gather(1, torch.tensor(r.token_ids)[:, None])[:, 0]
            assert float((gap / lg.std(-1)).max()) < 0.1


def test_synthetic_preset_decodes_and_matches_its_steps():
    """Random-init preset (GEMV shapes): the captured decode loop's history equals single steps' argmax."""
    from aios_amd.models.config import get_preset
    from aios_amd.runtime.loader import random_engine

    cfg = get_preset("test-gefazen")
    eng = random_engine(cfg, seed=3, max_ctx=256, max_slots=2, max_batch=2)
    ids = [int(t) for t in np.random.default_rng(0).integers(0, cfg.vocab_size, 30)]
    first = int(np.asarray(eng.prefill(0, ids, 0, True)).argmax())
    eng.decode_loop_prepare([0], [first], [30])
    eng.decode_loop_run(1, 40, True)
    hist = eng.decode_loop_history(1, 31, 40)
    lg = eng.step([1], [0], [30 + 40], ids + [first] + hist[:39], list(range(29, 70)))
    gap = lg.max(-1) - lg[np.arange(41), [first] + hist]
    assert float((gap / lg.std(-1)).max()) < 0.1
