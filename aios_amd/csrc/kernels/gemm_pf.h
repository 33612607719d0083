// Prefill GEMM on the CDNA4 matrix cores, dequantising the packed weights ONCE per workgroup tile:
//   C[M][N] (epilogue) = A[M][K] (bf16 activations) x W[N][K]^T (repacked Q4_K / Q6_K planes, or bf16)
// SURVEY.md §2.7 K3 prefill column -- the work llama.cpp's mul_mat_q does inside the reference's
// llama-server child (/root/reference/runtime/src/model_manager.rs:187-204) -- without any resident
// dequantised copy of a weight and without a vendor GEMM.
//
// Geometry (BM x BN tile, NW = BN / 32 waves): every wave owns ALL BM rows and 32 columns, i.e.
// (BM / 16) x 2 accumulators of v_mfma_f32_16x16x32_bf16.  A wave therefore dequantises exactly
// its own 32 columns' weights (each weight byte decoded once per workgroup, straight into MFMA B
// fragments in registers -- no bf16 LDS image of the weights, no LDS write pass) while the
// activation tile is shared by all waves through LDS.  Per 64-deep K-step a lane decodes 32
// weights (one 8-byte code group of each of its two columns) against 2 x BM/16 MFMAs.
//
// Staging: one LDS slot per K-step holds the A tile (BM rows x 128 B, 16-B units XOR-swizzled by
// row so a ds_read_b128 lane group of 16 rows hits 16 distinct bank slots) and the tile's raw
// weight bytes of that K-step (codes + per-format metadata), all moved by global_load_lds
// (LDS-DMA: no VGPR staging, no ds_write).  NS slots, NS - 1 K-steps in flight, one raw s_barrier
// per K-step (in-flight LDS-DMA survives it), counted s_waitcnt vmcnt -- the only vector-memory
// operations inside the loop are these DMAs, so the counts are exact (CDNA guide §5 "Pipelining
// across barriers", "Three .s-level traps").
//
// Weight k order: chunk h (16 B) of a 64-weight Q4_K group holds weights 16h + i (low nibble of byte
// i) and 32 + 16h + i (high nibble).  Lane quarter q of the 16x16x32 B fragment reads bytes
// 8(q&1) .. 8(q&1)+7 of chunk q>>1: its low nibbles are k = 8q .. 8q+7 (fragment of k-substep 0)
// and its high nibbles k = 32 + 8q .. (substep 1) -- exactly the MFMA's natural k layout, so the A
// fragments are plain 16-B row reads at unit 4s + q.  Q6_K is repacked into the same chunk order
// (qweight.h), its 2 high bits and int8 sub-block scales riding beside the codes.
#pragma once
#include <cstdlib>

#include "gemm_common.h"
#include "lds_dma.h"

namespace aios {

// GEPI_QKV (prefill chunks, non-NeoX RoPE, no QK-norm / bias, S = 1): the accumulator element
// (m, n) of this lane goes to the attention inputs directly -- RoPE'd q fp32 to q_out[m][q_dim], RoPE'd
// k and v as bf16 into the paged KV cache at (slot[m], pos[m]) -- the qkv_post launch and the fp32
// QKV round trip folded into the epilogue.  The RoPE partner (column n ^ 1) is the lane ^ 1 in both
// accumulator layouts (column = lane mod 16 / 32); every lane runs the DPP, the even one stores the pair.
__device__ __forceinline__ void pf_qkv_out(const GemmQArgs& a, int m, int n, float v, bool even) {
  const float w = __int_as_float(__builtin_amdgcn_mov_dpp(__float_as_int(v), 0xB1, 0xF, 0xF, false));
  if (!even || m >= a.M) return;
  const int hd = a.head_dim, pos = a.pos[m], slot = a.slot ? a.slot[m] : 0;
  float v0 = v, v1 = w;
  const int part = n < a.q_dim ? 0 : (n < a.q_dim + a.kv_dim ? 1 : 2);
  const int r = n - (part == 0 ? 0 : (part == 1 ? a.q_dim : a.q_dim + a.kv_dim));
  const int head = r / hd, lr = r - head * hd;
  if (part < 2) {
    const float2 t = a.rope_cs[(size_t)pos * (hd >> 1) + (lr >> 1)];
    const float o0 = v0 * t.x - v1 * t.y, o1 = v0 * t.y + v1 * t.x;
    v0 = o0;
    v1 = o1;
  }
  if (part == 0) {
    *(float2*)(a.q_out + (size_t)m * a.q_dim + n) = make_float2(v0, v1);
  } else {
    bf16_t* cache = part == 1 ? a.k_cache : a.v_cache;
    const size_t base = kv_offset(a.block_table, a.max_ctx / KV_BLOCK, slot, a.n_kv_heads, head, pos, hd);
    *(uint32_t*)(cache + base + lr) = pk_bf16(v0, v1);
  }
}


// slot layout for one K-step: A, then the weight planes of BN columns
template <int QT, int BM, int BN>
struct PfLayout {
  static constexpr bool Q6 = QT == QT_Q6_K, BF = QT == QT_BF16;
  static constexpr int A_BYTES = BM * 128;
  static constexpr int CODE = BF ? BN * 128 : BN * 32;        // bf16 rows (swizzled as A) / 2 code chunks
  static constexpr int META = BF ? 0 : BN * 16;                // Q4_K scale record / Q6_K high bits of 2 chunks
  static constexpr int SC = Q6 ? BN * 4 : 0;                   // Q6_K int8 scale pairs of the 2 chunks
  static constexpr int DW = Q6 ? BN * 4 : 0;                   // Q6_K aligned dword holding the block's f16 d
  static constexpr int OFF_CODE = A_BYTES, OFF_META = OFF_CODE + CODE, OFF_SC = OFF_META + META,
                       OFF_D = OFF_SC + SC;
  static constexpr int SLOT = (OFF_D + DW + 255) / 256 * 256;
  // DMA wave-instructions per slot: 1 KB at 16 B per lane, 256 B at 4 B per lane
  static constexpr int NI_A = A_BYTES / 1024, NI_CODE = CODE / 1024, NI_META = META / 1024, NI_SC = SC / 256,
                       NI_D = DW / 256;
  static constexpr int TI = NI_A + NI_CODE + NI_META + NI_SC + NI_D;
  static_assert(A_BYTES % 1024 == 0 && CODE % 1024 == 0 && META % 1024 == 0 && SC % 256 == 0, "slot pieces");
};

// This wave's share of every slot: pieces i = pp * NW + wv (pp < PH; the last may not exist).  The
// per-lane part of each piece's source address is a 32-bit byte offset computed once per workgroup;
// a K-step adds only a uniform per-kind step offset (the repacked planes advance linearly in kt:
// codes 32 B, Q6_K high bits 16 B, Q6_K scales 4 B per K-step; the 256-block records per 4 steps).
template <int QT, int BM, int BN, int NW>
struct PfDma {
  using L = PfLayout<QT, BM, BN>;
  static constexpr int PH = (L::TI + NW - 1) / NW;
  uint32_t off[PH];

  __device__ __forceinline__ void init(const GemmQArgs& a, int wrow0, int m0, int wv) {
    const int lane = threadIdx.x & 63;
    const uint32_t nbk = (uint32_t)a.K >> 8;
    static_for<PH>([&](auto ppc) {
      constexpr int pp = decltype(ppc)::value;
      int j = pp * NW + wv;
      uint32_t o = 0;
      if (j < L::NI_A) {  // A unit p -> row p>>3, logical 16-B unit (p&7) ^ ((row>>1)&7); rows past M re-read M-1
        const int p = 64 * j + lane, row = p >> 3, c = (p & 7) ^ ((row >> 1) & 7);
        const int m = min(m0 + row, a.M - 1);
        o = ((uint32_t)m * (uint32_t)a.lda + (uint32_t)(c * 8)) * 2u;
      } else if ((j -= L::NI_A) < L::NI_CODE) {
        const int p = 64 * j + lane;
        if constexpr (L::BF) {  // bf16 weight rows in the A swizzle
          const int col = p >> 3, c = (p & 7) ^ ((col >> 1) & 7);
          o = ((uint32_t)(wrow0 + col) * (uint32_t)a.K + (uint32_t)(c * 8)) * 2u;
        } else {  // column col's two 16-B code chunks (2g, 2g+1): 32 contiguous bytes
          const int col = p >> 1, h = p & 1;
          o = (uint32_t)(wrow0 + col) * nbk * 128u + (uint32_t)h * 16u;
        }
      } else if ((j -= L::NI_CODE) < L::NI_META) {
        const uint32_t row = (uint32_t)(wrow0 + 64 * j + lane);
        o = L::Q6 ? row * nbk * 64u : row * nbk * 16u;  // Q6_K high bits (8 B per chunk) / Q4_K record
      } else if ((j -= L::NI_META) < L::NI_SC) {
        o = (uint32_t)(wrow0 + 64 * j + lane) * nbk * 16u;  // Q6_K int8 scales (2 B per chunk)
      } else {
        j -= L::NI_SC;
        o = (uint32_t)(wrow0 + 64 * j + lane) * nbk;  // Q6_K d: the row's first block index
      }
      off[pp] = o;
    });
  }

  // issue K-step kt into dst (all of this wave's pieces, or those with pp % NP == P: spread over phases)
  template <int P = 0, int NP = 1>
  __device__ __forceinline__ void issue(const GemmQArgs& a, const QWeight& w, int kt, uint32_t dst, int wv) const {
    static_for<PH>([&](auto ppc) {
      constexpr int pp = decltype(ppc)::value;
      if constexpr (pp % NP != P) return;
      int j = pp * NW + wv;
      if (j >= L::TI) return;
      if (j < L::NI_A) {
        const uint8_t* src = (const uint8_t*)a.A + kt * 128 + off[pp];
        pf_glds16(src, dst + j * 1024);
      } else if ((j -= L::NI_A) < L::NI_CODE) {
        const uint8_t* src = w.p0 + (L::BF ? kt * 128 : kt * 32) + off[pp];
        pf_glds16(src, dst + L::OFF_CODE + j * 1024);
      } else if ((j -= L::NI_CODE) < L::NI_META) {
        const uint8_t* src = w.p1 + (L::Q6 ? kt * 16 : (kt >> 2) * 16) + off[pp];
        pf_glds16(src, dst + L::OFF_META + j * 1024);
      } else if ((j -= L::NI_META) < L::NI_SC) {
        const uint8_t* src = w.p2 + kt * 4 + off[pp];
        pf_glds4(src, dst + L::OFF_SC + j * 256);
      } else {
        j -= L::NI_SC;
        const uint8_t* src = w.p3 + (((off[pp] + (uint32_t)(kt >> 2)) >> 1) << 2);  // the dword holding f16 d
        pf_glds4(src, dst + L::OFF_D + j * 256);
      }
    });
  }
};

// 8 codes (bytes of w0 then w1) -> bf16x8 fragment of sc * q - of
__device__ __forceinline__ gbf16x8 pf_dq8(uint32_t w0, uint32_t w1, float sc, float of) {
  asm volatile("" : "+v"(w0), "+v"(w1));  // one v_cvt_f32_ubyteN per byte
  uint32_t p[4];
  p[0] = pk_bf16(fmaf(sc, (float)(w0 & 0xff), -of), fmaf(sc, (float)((w0 >> 8) & 0xff), -of));
  p[1] = pk_bf16(fmaf(sc, (float)((w0 >> 16) & 0xff), -of), fmaf(sc, (float)(w0 >> 24), -of));
  p[2] = pk_bf16(fmaf(sc, (float)(w1 & 0xff), -of), fmaf(sc, (float)((w1 >> 8) & 0xff), -of));
  p[3] = pk_bf16(fmaf(sc, (float)((w1 >> 16) & 0xff), -of), fmaf(sc, (float)(w1 >> 24), -of));
  gbf16x8 r;
  __builtin_memcpy(&r, p, 16);
  return r;
}

// Raw weight bytes of one tile column for this lane's quarter q (LDS reads), then the decode of
// fragment s (k 8q.. for s = 0, 32 + 8q.. for s = 1) -- split so the decode can sit between MFMAs.
struct PfBRaw {
  uint2 cw;       // 8 code bytes: low nibbles = fragment 0, high nibbles = fragment 1
  uint4 mt;       // Q4_K scale record | bf16: fragment 0
  uint2 hb;       // Q6_K high bits {run 0, run 1}
  uint32_t scw;   // Q6_K int8 scale pairs
  uint32_t dw;    // Q6_K dword holding d
  uint4 b1;       // bf16: fragment 1
};

template <int QT, int BM, int BN>
__device__ __forceinline__ void pf_braw(const uint8_t* slot, int col, int q, PfBRaw& r) {
  using L = PfLayout<QT, BM, BN>;
  if constexpr (L::BF) {
    r.mt = *(const uint4*)(slot + L::OFF_CODE + col * 128 + (((0 + q) ^ ((col >> 1) & 7)) << 4));
    r.b1 = *(const uint4*)(slot + L::OFF_CODE + col * 128 + (((4 + q) ^ ((col >> 1) & 7)) << 4));
  } else {
    r.cw = *(const uint2*)(slot + L::OFF_CODE + col * 32 + 8 * q);
    if constexpr (L::Q6) {
      r.hb = *(const uint2*)(slot + L::OFF_META + col * 16 + 8 * (q >> 1));
      r.scw = *(const uint32_t*)(slot + L::OFF_SC + col * 4);
      r.dw = *(const uint32_t*)(slot + L::OFF_D + col * 4);
    } else {
      r.mt = *(const uint4*)(slot + L::OFF_META + col * 16);
    }
  }
}

template <int QT, int S>
__device__ __forceinline__ gbf16x8 pf_bdec(const PfBRaw& r, int q, int kt, int dpar) {
  gbf16x8 f;
  if constexpr (QT == QT_BF16) {
    const uint4 v = S == 0 ? r.mt : r.b1;
    __builtin_memcpy(&f, &v, 16);
  } else if constexpr (QT == QT_Q8_0) {  // (pf8 body) fragment S = the K-step's 32-block S: cw / b1.xy
    const uint32_t w0 = (S == 0 ? r.cw.x : r.b1.x) ^ 0x80808080u, w1 = (S == 0 ? r.cw.y : r.b1.y) ^ 0x80808080u;
    const float d = h2f((uint16_t)(r.scw >> (16 * S)));
    f = pf_dq8(w0, w1, d, 128.f * d);
  } else if constexpr (QT == QT_Q4_0) {  // block S: weights 8q.. = low nibbles (q < 2) / high (q >= 2)
    const int sh = 4 * (q >> 1);
    const uint32_t w0 = ((S == 0 ? r.cw.x : r.b1.x) >> sh) & 0x0f0f0f0fu, w1 = ((S == 0 ? r.cw.y : r.b1.y) >> sh) & 0x0f0f0f0fu;
    const float d = h2f((uint16_t)(r.scw >> (16 * S)));
    f = pf_dq8(w0, w1, d, 8.f * d);
  } else if constexpr (QT == QT_Q6_K) {
    const float d = h2f((uint16_t)(r.dw >> (16 * dpar)));
    const float ds = d * (float)(int8_t)((r.scw >> (16 * (q >> 1) + 8 * S)) & 0xff);
    const uint32_t hv = S == 0 ? r.hb.x : r.hb.y;
    const int j0 = 2 * (q & 1);  // code words j0, j0 + 1 of the chunk
    const uint32_t c0 = S == 0 ? (r.cw.x & 0x0f0f0f0fu) : ((r.cw.x >> 4) & 0x0f0f0f0fu);
    const uint32_t c1 = S == 0 ? (r.cw.y & 0x0f0f0f0fu) : ((r.cw.y >> 4) & 0x0f0f0f0fu);
    f = pf_dq8(c0 | (((hv >> (2 * j0)) & 0x03030303u) << 4), c1 | (((hv >> (2 * j0 + 2)) & 0x03030303u) << 4), ds,
               32.f * ds);
  } else {  // Q4_K
    const float d = h2f((uint16_t)(r.mt.x & 0xffff)), dmin = h2f((uint16_t)(r.mt.x >> 16));
    const uint32_t fl = kq_field(r.mt.y, r.mt.z, r.mt.w, kt & 3);
    const float ds = d * (float)((fl >> (6 * S)) & 63), dm = dmin * (float)((fl >> (12 + 6 * S)) & 63);
    uint32_t c0 = S == 0 ? (r.cw.x & 0x0f0f0f0fu) : ((r.cw.x >> 4) & 0x0f0f0f0fu);
    uint32_t c1 = S == 0 ? (r.cw.y & 0x0f0f0f0fu) : ((r.cw.y >> 4) & 0x0f0f0f0fu);
    if constexpr (QT == QT_Q5_K) {  // (pf8 body) qh bytes 8q.. in hb: bit 2g + S
      const int sh = 2 * (kt & 3) + S;
      c0 |= ((r.hb.x >> sh) & 0x01010101u) << 4;
      c1 |= ((r.hb.y >> sh) & 0x01010101u) << 4;
    }
    f = pf_dq8(c0, c1, ds, dm);
  }
  return f;
}

// PROBE (timing anatomy only, tools/bench_gemm.py --pf-probe; never in the engine's launches):
// 1 = no DMA waits, 4 = no DMA issued inside the loop (stale slots), 8 = no per-step barrier
template <int QT, int BM, int NW, int NS, int EPI, int PROBE = 0>
__device__ __forceinline__ void pf_body(const GemmQArgs& a, int m0, int n0, int seg, int kt0, int kt1, int S) {
  constexpr int BN = NW * 32, MT = BM / 16;
  constexpr int GR = MT < 8 ? MT : 8, NG = MT / GR;  // row tiles per phase, phases per k-substep
  using L = PfLayout<QT, BM, BN>;
  extern __shared__ __attribute__((aligned(16))) uint8_t pf_smem[];
  const int tid = threadIdx.x, lane = tid & 63;
  const int wv = __builtin_amdgcn_readfirstlane(tid >> 6);
  QWeight w;  // field-wise uniform selects (a dynamically indexed struct copy goes to scratch)
  w.qtype = QT;
  w.rows = seg == 0 ? a.seg[0].rows : (seg == 1 ? a.seg[1].rows : a.seg[2].rows);
  w.cols = a.K;
  w.pad_ = 0;
  w.p0 = seg == 0 ? a.seg[0].p0 : (seg == 1 ? a.seg[1].p0 : a.seg[2].p0);
  w.p1 = seg == 0 ? a.seg[0].p1 : (seg == 1 ? a.seg[1].p1 : a.seg[2].p1);
  w.p2 = seg == 0 ? a.seg[0].p2 : (seg == 1 ? a.seg[1].p2 : a.seg[2].p2);
  w.p3 = seg == 0 ? a.seg[0].p3 : (seg == 1 ? a.seg[1].p3 : a.seg[2].p3);
  const int wrow0 = n0 - (seg == 0 ? a.seg_n0[0] : (seg == 1 ? a.seg_n0[1] : a.seg_n0[2]));
  const int nbk = a.K >> 8;
  const int r16 = lane & 15, q = lane >> 4;
  const int col0 = wv * 32 + r16;  // this lane's two columns: col0, col0 + 16 (tile-relative)

  gf32x4 acc[MT][2];
#pragma unroll
  for (int i = 0; i < MT; ++i)
#pragma unroll
    for (int c = 0; c < 2; ++c) acc[i][c] = gf32x4{0.f, 0.f, 0.f, 0.f};

  // pieces per slot of this wave (PH if wv < TI % NW): the vmcnt immediates
  constexpr int PH = (L::TI + NW - 1) / NW, PLO = L::TI / NW;
  const bool many = (L::TI % NW == 0) || wv < L::TI % NW;
  const int nk = kt1 - kt0;
  PfDma<QT, BM, BN, NW> dma;
  const uint32_t lds0 = __builtin_amdgcn_readfirstlane(pf_lds_addr(pf_smem));
  dma.init(a, wrow0, m0, wv);
#pragma unroll
  for (int p = 0; p < NS - 1; ++p)
    if (p < nk) dma.issue(a, w, kt0 + p, lds0 + p * L::SLOT, wv);

  int cur = 0;
  for (int t = 0; t < nk; ++t) {
    // step t's pieces landed (the younger NS - 2 steps may stay in flight), then everyone's
    if constexpr (PROBE & 1) {
    } else if constexpr (NS == 3) {
      if (t + 1 < nk) {
        if (many) pf_vmcnt<PH>(); else pf_vmcnt<PLO>();
      } else {
        pf_vmcnt<0>();
      }
    } else {
      static_assert(NS == 2, "2 or 3 slots");
      pf_vmcnt<0>();
    }
    if constexpr (!(PROBE & 8)) pf_barrier();
    // refill the slot every wave finished reading last step
    if (!(PROBE & 4) && t + NS - 1 < nk) {
      const int ns = cur == 0 ? NS - 1 : cur - 1;
      dma.issue(a, w, kt0 + t + NS - 1, lds0 + ns * L::SLOT, wv);
    }
    const uint8_t* slot = pf_smem + cur * L::SLOT;
    const int kt = kt0 + t;
    // Phases: A fragments of GR row tiles per phase in two named register groups (fa / fb), the
    // next phase's reads issued before this phase's MFMAs; fragment-1 decode inside phase 0.
    // sched_barrier pins the phase order (hipcc otherwise keeps ~2 reads in flight per MFMA pair).
    PfBRaw raw[2];
    int dpar[2];
#pragma unroll
    for (int c = 0; c < 2; ++c) {
      const int col = col0 + 16 * c;
      dpar[c] = L::Q6 ? (int)(((uint32_t)(wrow0 + col) * (uint32_t)nbk + (uint32_t)(kt >> 2)) & 1u) : 0;
      pf_braw<QT, BM, BN>(slot, col, q, raw[c]);
    }
    gbf16x8 fa[GR], fb[GR], bf[2][2];
    auto ldA = [&](gbf16x8(&f)[GR], int p) __attribute__((always_inline)) {
      const int sp = p / NG, g = p % NG;
#pragma unroll
      for (int i = 0; i < GR; ++i) {
        const int row = 16 * (g * GR + i) + r16;
        const uint4 av = *(const uint4*)(slot + row * 128 + (((4 * sp + q) ^ ((row >> 1) & 7)) << 4));
        __builtin_memcpy(&f[i], &av, 16);
      }
    };
    ldA(fa, 0);
    __builtin_amdgcn_sched_barrier(0);  // every read of the step's head in flight before the decode
#pragma unroll
    for (int c = 0; c < 2; ++c) bf[c][0] = pf_bdec<QT, 0>(raw[c], q, kt, dpar[c]);
    __builtin_amdgcn_sched_barrier(0);
    static_for<2 * NG>([&](auto pc) {
      constexpr int p = decltype(pc)::value, sp = p / NG, g = p % NG;
      if constexpr (p + 1 < 2 * NG) {
        if constexpr (p % 2 == 0) ldA(fb, p + 1);
        else ldA(fa, p + 1);
      }
      if constexpr (p == 0) {
#pragma unroll
        for (int c = 0; c < 2; ++c) bf[c][1] = pf_bdec<QT, 1>(raw[c], q, kt, dpar[c]);
      }
#pragma unroll
      for (int i = 0; i < GR; ++i)
#pragma unroll
        for (int c = 0; c < 2; ++c)
          acc[g * GR + i][c] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(p % 2 == 0 ? fa[i] : fb[i], bf[c][sp],
                                                                       acc[g * GR + i][c], 0, 0, 0);
      __builtin_amdgcn_sched_barrier(0);
    });
    asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");  // this slot's LDS reads retired before it is refilled
    cur = cur == NS - 1 ? 0 : cur + 1;
  }

  // epilogue -- C/D map of the 16x16 accumulator: col = lane & 15, row = 4 * (lane >> 4) + e
#pragma unroll
  for (int c = 0; c < 2; ++c) {
    const int n = n0 + col0 + 16 * c;
#pragma unroll
    for (int i = 0; i < MT; ++i) {
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const int m = m0 + 16 * i + 4 * q + e;
        const float v = acc[i][c][e];
        if constexpr (EPI == GEPI_SWIGLU_BF16) {
          // interleaved gate/up columns: even lane = gate, odd lane = its up partner
          const float up = __int_as_float(__builtin_amdgcn_mov_dpp(__float_as_int(v), 0xB1, 0xF, 0xF, false));
          if (m < a.M && !(r16 & 1)) a.C16[(size_t)m * a.ldc + (n >> 1)] = f32_to_bf16(glu_act(v, a.act) * up);
        } else if constexpr (EPI == GEPI_STORE16) {
          if (m < a.M) a.C16[(size_t)m * a.ldc + n] = f32_to_bf16(store16_val(a, n, v));
        } else if constexpr (EPI == GEPI_QKV) {
          pf_qkv_out(a, m, n, v, !(r16 & 1));
        } else if (m < a.M) {
          float* cp = a.C + (size_t)m * a.ldc + n;
          if (S > 1) unsafeAtomicAdd(cp, v);
          else if constexpr (EPI == GEPI_ACCUM) *cp += v;
          else *cp = v;
        }
      }
    }
  }
}


// ---- 32x32x16 body: a wave owns BM rows x 32 columns = BM/32 accumulators of v_mfma_f32_32x32x16_bf16.
// Per 64-deep K-step four k16 substeps s = 0..3 at k = 16s + 8h + j (h = lane >> 5): chunk (s & 1)'s
// bytes 8h .. 8h+7, low nibbles for s < 2, high nibbles for s >= 2 -- again the MFMA's natural k
// layout, so A fragments are 16-B row reads at unit 2s + h.  Per MFMA (32 cycles, vector issue held
// for 8) there is room for ~6 fillers against ~2 on the 16x16x32 body, which left that body
// issue-bound on its decode VALU + LDS reads (tools/bench_gemm.py --pf-probe, round 5).  The slot's
// DMA pieces are issued one phase at a time between the MFMA groups instead of at the step head.
struct PfBRaw32 {
  uint2 c0, c1;   // 8 code bytes of chunk 0 / chunk 1
  uint4 mt;       // Q4_K scale record | Q6_K high bits {c0 run0, c0 run1, c1 run0, c1 run1} | bf16 fragment 0
  uint32_t scw;   // Q6_K int8 scales {c0 run0, c0 run1, c1 run0, c1 run1}
  uint32_t dw;    // Q6_K dword holding d
  uint4 b1, b2, b3;  // bf16 fragments 1..3
};

template <int QT, int BM, int BN>
__device__ __forceinline__ void pf_braw32(const uint8_t* slot, int col, int h, PfBRaw32& r) {
  using L = PfLayout<QT, BM, BN>;
  if constexpr (L::BF) {
    const uint8_t* row = slot + L::OFF_CODE + col * 128;
    const int x = (col >> 1) & 7;
    r.mt = *(const uint4*)(row + (((0 + h) ^ x) << 4));
    r.b1 = *(const uint4*)(row + (((2 + h) ^ x) << 4));
    r.b2 = *(const uint4*)(row + (((4 + h) ^ x) << 4));
    r.b3 = *(const uint4*)(row + (((6 + h) ^ x) << 4));
  } else {
    r.c0 = *(const uint2*)(slot + L::OFF_CODE + col * 32 + 8 * h);
    r.c1 = *(const uint2*)(slot + L::OFF_CODE + col * 32 + 16 + 8 * h);
    r.mt = *(const uint4*)(slot + L::OFF_META + col * 16);
    if constexpr (L::Q6) {
      r.scw = *(const uint32_t*)(slot + L::OFF_SC + col * 4);
      r.dw = *(const uint32_t*)(slot + L::OFF_D + col * 4);
    }
  }
}

template <int QT, int S>
__device__ __forceinline__ gbf16x8 pf_bdec32(const PfBRaw32& r, int h, int kt, int dpar) {
  gbf16x8 f;
  if constexpr (QT == QT_BF16) {
    const uint4 v = S == 0 ? r.mt : (S == 1 ? r.b1 : (S == 2 ? r.b2 : r.b3));
    __builtin_memcpy(&f, &v, 16);
  } else if constexpr (QT == QT_Q8_0) {  // int8 codes (+128 -> the unsigned decode), d of block S >> 1
    const uint32_t w0 = (S == 0 ? r.c0.x : (S == 1 ? r.c1.x : (S == 2 ? r.b1.x : r.b1.z))) ^ 0x80808080u;
    const uint32_t w1 = (S == 0 ? r.c0.y : (S == 1 ? r.c1.y : (S == 2 ? r.b1.y : r.b1.w))) ^ 0x80808080u;
    const float d = h2f((uint16_t)(r.scw >> (16 * (S >> 1))));
    f = pf_dq8(w0, w1, d, 128.f * d);
  } else if constexpr (QT == QT_Q4_0) {  // block S >> 1: low nibbles = weights 0..15, high = 16..31
    const uint2 cw = (S >> 1) ? r.c1 : r.c0;
    const uint32_t w0 = (S & 1) ? ((cw.x >> 4) & 0x0f0f0f0fu) : (cw.x & 0x0f0f0f0fu);
    const uint32_t w1 = (S & 1) ? ((cw.y >> 4) & 0x0f0f0f0fu) : (cw.y & 0x0f0f0f0fu);
    const float d = h2f((uint16_t)(r.scw >> (16 * (S >> 1))));
    f = pf_dq8(w0, w1, d, 8.f * d);
  } else {
    const uint2 cw = (S & 1) ? r.c1 : r.c0;
    const uint32_t w0 = (S < 2) ? (cw.x & 0x0f0f0f0fu) : ((cw.x >> 4) & 0x0f0f0f0fu);
    const uint32_t w1 = (S < 2) ? (cw.y & 0x0f0f0f0fu) : ((cw.y >> 4) & 0x0f0f0f0fu);
    if constexpr (QT == QT_Q6_K) {
      // run (S >> 1) of chunk (S & 1): high-bit word and int8 scale
      constexpr int idx = 2 * (S & 1) + (S >> 1);
      const uint32_t hv = idx == 0 ? r.mt.x : (idx == 1 ? r.mt.y : (idx == 2 ? r.mt.z : r.mt.w));
      const float d = h2f((uint16_t)(r.dw >> (16 * dpar)));
      const float ds = d * (float)(int8_t)((r.scw >> (8 * idx)) & 0xff);
      const int j0 = 2 * h;  // code words 2h, 2h + 1 of the chunk
      f = pf_dq8(w0 | (((hv >> (2 * j0)) & 0x03030303u) << 4), w1 | (((hv >> (2 * j0 + 2)) & 0x03030303u) << 4), ds,
                 32.f * ds);
    } else {  // Q4_K / Q5_K: sub-block 2g (S < 2) or 2g + 1
      const float d = h2f((uint16_t)(r.mt.x & 0xffff)), dmin = h2f((uint16_t)(r.mt.x >> 16));
      const uint32_t fl = kq_field(r.mt.y, r.mt.z, r.mt.w, kt & 3);
      constexpr int sb = S >> 1;
      const float ds = d * (float)((fl >> (6 * sb)) & 63), dm = dmin * (float)((fl >> (12 + 6 * sb)) & 63);
      if constexpr (QT == QT_Q5_K) {  // + bit (2g + hi) of the weights' qh bytes as bit 4
        const int sh = 2 * (kt & 3) + sb;
        const uint32_t h0 = (S & 1) ? r.b1.z : r.b1.x, h1 = (S & 1) ? r.b1.w : r.b1.y;
        f = pf_dq8(w0 | (((h0 >> sh) & 0x01010101u) << 4), w1 | (((h1 >> sh) & 0x01010101u) << 4), ds, dm);
      } else {
        f = pf_dq8(w0, w1, ds, dm);
      }
    }
  }
  return f;
}

template <int QT, int BM, int NW, int NS, int EPI, int PROBE = 0>
__device__ __forceinline__ void pf_body32(const GemmQArgs& a, int m0, int n0, int seg, int kt0, int kt1, int S) {
  constexpr int BN = NW * 32, MT = BM / 32;
  using L = PfLayout<QT, BM, BN>;
  extern __shared__ __attribute__((aligned(16))) uint8_t pf_smem[];
  const int tid = threadIdx.x, lane = tid & 63;
  const int wv = __builtin_amdgcn_readfirstlane(tid >> 6);
  QWeight w;
  w.qtype = QT;
  w.rows = seg == 0 ? a.seg[0].rows : (seg == 1 ? a.seg[1].rows : a.seg[2].rows);
  w.cols = a.K;
  w.pad_ = 0;
  w.p0 = seg == 0 ? a.seg[0].p0 : (seg == 1 ? a.seg[1].p0 : a.seg[2].p0);
  w.p1 = seg == 0 ? a.seg[0].p1 : (seg == 1 ? a.seg[1].p1 : a.seg[2].p1);
  w.p2 = seg == 0 ? a.seg[0].p2 : (seg == 1 ? a.seg[1].p2 : a.seg[2].p2);
  w.p3 = seg == 0 ? a.seg[0].p3 : (seg == 1 ? a.seg[1].p3 : a.seg[2].p3);
  const int wrow0 = n0 - (seg == 0 ? a.seg_n0[0] : (seg == 1 ? a.seg_n0[1] : a.seg_n0[2]));
  const int nbk = a.K >> 8;
  const int r32 = lane & 31, h = lane >> 5;
  const int col = wv * 32 + r32;  // this lane's tile column

  gf32x16 acc[MT];
#pragma unroll
  for (int i = 0; i < MT; ++i)
#pragma unroll
    for (int e = 0; e < 16; ++e) acc[i][e] = 0.f;

  constexpr int PH = (L::TI + NW - 1) / NW, PLO = L::TI / NW;
  const bool many = (L::TI % NW == 0) || wv < L::TI % NW;
  const int nk = kt1 - kt0;
  PfDma<QT, BM, BN, NW> dma;
  const uint32_t lds0 = __builtin_amdgcn_readfirstlane(pf_lds_addr(pf_smem));
  dma.init(a, wrow0, m0, wv);
#pragma unroll
  for (int p = 0; p < NS - 1; ++p)
    if (p < nk) dma.issue(a, w, kt0 + p, lds0 + p * L::SLOT, wv);

  int cur = 0;
  for (int t = 0; t < nk; ++t) {
    if constexpr (PROBE & 1) {
    } else if constexpr (NS == 3) {
      if (t + 1 < nk) {
        if (many) pf_vmcnt<PH>(); else pf_vmcnt<PLO>();
      } else {
        pf_vmcnt<0>();
      }
    } else {
      static_assert(NS == 2, "2 or 3 slots");
      pf_vmcnt<0>();
    }
    if constexpr (!(PROBE & 8)) pf_barrier();
    const bool refill = !(PROBE & 4) && t + NS - 1 < nk;
    const uint32_t nslot = lds0 + (cur == 0 ? NS - 1 : cur - 1) * L::SLOT;
    const int knext = kt0 + t + NS - 1;
    const uint8_t* slot = pf_smem + cur * L::SLOT;
    const int kt = kt0 + t;
    const int dpar = L::Q6 ? (int)(((uint32_t)(wrow0 + col) * (uint32_t)nbk + (uint32_t)(kt >> 2)) & 1u) : 0;
    PfBRaw32 raw;
    pf_braw32<QT, BM, BN>(slot, col, h, raw);
    gbf16x8 fa[MT], fb[MT], bf[4];
    auto ldA = [&](gbf16x8(&f)[MT], int sp) __attribute__((always_inline)) {
#pragma unroll
      for (int i = 0; i < MT; ++i) {
        const int row = 32 * i + r32;
        const uint4 av = *(const uint4*)(slot + row * 128 + (((2 * sp + h) ^ ((row >> 1) & 7)) << 4));
        __builtin_memcpy(&f[i], &av, 16);
      }
    };
    ldA(fa, 0);
    __builtin_amdgcn_sched_barrier(0);
    bf[0] = pf_bdec32<QT, 0>(raw, h, kt, dpar);
    __builtin_amdgcn_sched_barrier(0);
    // phase sp: next substep's A reads, one share of the refill DMA, the next fragment's decode, the MFMAs
    static_for<4>([&](auto pc) {
      constexpr int sp = decltype(pc)::value;
      if constexpr (sp + 1 < 4) {
        if constexpr (sp % 2 == 0) ldA(fb, sp + 1);
        else ldA(fa, sp + 1);
      }
      if (refill) dma.template issue<sp, 4>(a, w, knext, nslot, wv);
      if constexpr (sp + 1 < 4) bf[sp + 1] = pf_bdec32<QT, sp + 1>(raw, h, kt, dpar);
#pragma unroll
      for (int i = 0; i < MT; ++i)
        acc[i] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(sp % 2 == 0 ? fa[i] : fb[i], bf[sp], acc[i], 0, 0, 0);
      __builtin_amdgcn_sched_barrier(0);
    });
    asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
    cur = cur == NS - 1 ? 0 : cur + 1;
  }

  // epilogue -- C/D map of the 32x32 accumulator: col = lane & 31, row = (e & 3) + 8 (e >> 2) + 4 h
  const int n = n0 + col;
#pragma unroll
  for (int i = 0; i < MT; ++i) {
#pragma unroll
    for (int e = 0; e < 16; ++e) {
      const int m = m0 + 32 * i + (e & 3) + 8 * (e >> 2) + 4 * h;
      const float v = acc[i][e];
      if constexpr (EPI == GEPI_SWIGLU_BF16) {
        const float up = __int_as_float(__builtin_amdgcn_mov_dpp(__float_as_int(v), 0xB1, 0xF, 0xF, false));
        if (m < a.M && !(r32 & 1)) a.C16[(size_t)m * a.ldc + (n >> 1)] = f32_to_bf16(glu_act(v, a.act) * up);
      } else if constexpr (EPI == GEPI_STORE16) {
        if (m < a.M) a.C16[(size_t)m * a.ldc + n] = f32_to_bf16(store16_val(a, n, v));
      } else if (m < a.M) {
        float* cp = a.C + (size_t)m * a.ldc + n;
        if (S > 1) unsafeAtomicAdd(cp, v);
        else if constexpr (EPI == GEPI_ACCUM) *cp += v;
        else *cp = v;
      }
    }
  }
}


// ==== pf4: 4 waves (one per SIMD) x WC columns each, 32x32x16 MFMA, accumulators in AGPRs ============
// Round-5 probes (tools/bench_gemm.py --pf-probe + rocprofv3 PMC, gate/up M = 2048): with 8 waves the
// two waves of a SIMD race for its matrix pipe, the leader then idles at every per-step barrier
// (SQ_WAIT_ANY 148M vs 55M quad-cycles without the barrier) while the step head -- fragment reads
// and the B decode -- ran with the pipe idle; the runtime piece selection of the shared DMA added
// ~68 SALU per wave-step.  Here each wave owns its SIMD, DMAs its OWN weight columns (so it can
// wait for, read and decode step t+1's B fragments with its own vmcnt, before the barrier, inside
// step t's last phases) and every DMA piece is compile-time: one vmcnt immediate per wave.
//
// Formats beyond Q4_K / Q6_K / bf16 (round 6) read the GEMV engines' planes
// (quant_pack.hip) in place -- no second copy of any weight:
//   Q5_K  = the Q4_K codes + record, plus the block's 32 qh bytes (bit 2g + hi of byte l = high bit of
//           weight 64g + 32hi + l) fetched with every K-step as one more 1 KB piece;
//   Q4_0  = 32-weight blocks: the K-step's two 16-B code blocks (the Q4_K code reads, a different
//           nibble <-> fragment map) + the dword holding both blocks' f16 d (4-B piece, as Q6_K's scales);
//   Q8_0  = row-major int8 codes, 64 B per column per K-step (two 1 KB pieces) + the d-pair dword.
template <int QT>
struct PfFmt {
  static constexpr bool Q6 = QT == QT_Q6_K, BF = QT == QT_BF16, Q5 = QT == QT_Q5_K, L0 = QT == QT_Q4_0,
                        L8 = QT == QT_Q8_0, KREC = QT == QT_Q4_K || QT == QT_Q5_K;
};
#ifndef AIOS_PF4_NS
#define AIOS_PF4_NS 3
#endif
template <int QT, int BM, int WC, int NW = 4>
struct Pf4Layout {
  using F = PfFmt<QT>;
  static constexpr bool Q6 = F::Q6, BF = F::BF, Q5 = F::Q5, L0 = F::L0, L8 = F::L8;
  static constexpr int A_BYTES = BM * 128;
  // per wave: bf16 rows / Q8_0 bytes / 2 code chunks per column
  static constexpr int CODE = BF ? WC * 128 : (L8 ? WC * 64 : WC * 32);
  static constexpr int META = (F::KREC || Q6) ? (WC * 16 > 1024 ? WC * 16 : 1024) : 0;  // K record / Q6_K high bits
  static constexpr int HB = Q5 ? WC * 32 : 0;                                             // Q5_K qh bytes
  static constexpr int SC = (Q6 || L0 || L8) ? 256 : 0;  // Q6_K int8 scales / Q4_0, Q8_0 d pair (4-B pieces)
  static constexpr int DW = Q6 ? 256 : 0;                // Q6_K d dword
  static constexpr int OFF_META = CODE, OFF_HB = OFF_META + META, OFF_SC = OFF_HB + HB, OFF_DW = OFF_SC + SC;
  static constexpr int WB = OFF_DW + DW;                 // one wave's weight bytes per slot
  static constexpr int OFF_B = A_BYTES;
  static constexpr int SLOT = (A_BYTES + NW * WB + 255) / 256 * 256;
  // ring depth: as many slots as 160 KB of LDS holds, up to AIOS_PF4_NS (deeper rings keep more K-steps of
  // DMA in flight for the one workgroup per CU; the counted waits are (NS - 1) / (NS - 2) x PW)
  static constexpr int NS_FIT = (160 * 1024) / SLOT;
  static constexpr int NS = NS_FIT < AIOS_PF4_NS ? NS_FIT : AIOS_PF4_NS;
  static constexpr int NA = BM / (8 * NW), NCODE = CODE / 1024, NMETA = META / 1024, NHB = HB / 1024,
                       NSC = SC / 256, ND = DW / 256;
  static constexpr int PW = NA + NCODE + NMETA + NHB + NSC + ND;  // DMA instructions per wave per slot
  static_assert(CODE % 1024 == 0 && HB % 1024 == 0 && WC * 4 <= 256 && PW <= 31 && NA * 8 * NW == BM, "pf4 slot");
  static_assert(NS >= 2 && (NS - 1) * PW <= 63, "pf4 ring depth / vmcnt immediate");
};

template <int QT, int BM, int WC, int NW = 4>
struct Pf4Dma {
  using L = Pf4Layout<QT, BM, WC, NW>;
  uint32_t off[L::PW];

  __device__ __forceinline__ void init(const GemmQArgs& a, int wcol0, int m0, int wv) {
    const int lane = threadIdx.x & 63;
    const uint32_t nbk = (uint32_t)a.K >> 8;
    static_for<L::PW>([&](auto ic) {
      constexpr int i = decltype(ic)::value;
      uint32_t o;
      if constexpr (i < L::NA) {  // A piece j = NW i + wv: unit p -> row p>>3, logical unit (p&7) ^ ((row>>1)&7)
        const int p = 64 * (NW * i + wv) + lane, row = p >> 3, c = (p & 7) ^ ((row >> 1) & 7);
        const int m = min(m0 + row, a.M - 1);
        o = ((uint32_t)m * (uint32_t)a.lda + (uint32_t)(c * 8)) * 2u;
      } else if constexpr (i < L::NA + L::NCODE) {
        const int p = 64 * (i - L::NA) + lane;
        if constexpr (L::BF) {
          const int col = p >> 3, c = (p & 7) ^ ((col >> 1) & 7);
          o = ((uint32_t)(wcol0 + col) * (uint32_t)a.K + (uint32_t)(c * 8)) * 2u;
        } else if constexpr (L::L8) {  // 4 x 16 B per column
          const int col = p >> 2, u = p & 3;
          o = (uint32_t)(wcol0 + col) * nbk * 256u + (uint32_t)u * 16u;
        } else {
          const int col = p >> 1, hh = p & 1;
          o = (uint32_t)(wcol0 + col) * nbk * 128u + (uint32_t)hh * 16u;
        }
      } else if constexpr (i < L::NA + L::NCODE + L::NMETA) {
        const uint32_t row = (uint32_t)(wcol0 + (lane & (WC - 1)));
        o = L::Q6 ? row * nbk * 64u : row * nbk * 16u;
      } else if constexpr (i < L::NA + L::NCODE + L::NMETA + L::NHB) {  // Q5_K qh: 2 x 16 B per column
        o = (uint32_t)(wcol0 + (lane >> 1)) * nbk * 32u + (uint32_t)(lane & 1) * 16u;
      } else if constexpr (i < L::NA + L::NCODE + L::NMETA + L::NHB + L::NSC) {
        o = (uint32_t)(wcol0 + (lane & (WC - 1))) * nbk * 16u;  // (Q4_0 / Q8_0: K / 16 bytes of d per row)
      } else {
        o = (uint32_t)(wcol0 + (lane & (WC - 1))) * nbk;
      }
      off[i] = o;
    });
  }

  // K-step kt into the slot at LDS byte address dst (wave-uniform).  PROBE 16: weight pieces read
  // contiguous 1 KB (wrong data; coalescing probe), PROBE 32: no weight pieces (timing only)
  template <int PROBE = 0>
  __device__ __forceinline__ void issue(const GemmQArgs& a, const QWeight& w, int kt, uint32_t dst, int wv) const {
    const uint32_t wb = dst + L::OFF_B + (uint32_t)wv * L::WB;
    static_for<L::PW>([&](auto ic) {
      constexpr int i = decltype(ic)::value;
      if constexpr ((PROBE & 32) && i >= L::NA) return;
      if constexpr ((PROBE & 16) && i >= L::NA) {
        pf_glds16(w.p0 + kt * 4096 + (i - L::NA) * 1024 + (threadIdx.x & 63) * 16 + wv * 65536, wb + (i - L::NA) * 256);
        return;
      }
      if constexpr (i < L::NA) {
        pf_glds16((const uint8_t*)a.A + kt * 128 + off[i], dst + (NW * i + wv) * 1024);
      } else if constexpr (i < L::NA + L::NCODE) {
        pf_glds16(w.p0 + (L::BF ? kt * 128 : (L::L8 ? kt * 64 : kt * 32)) + off[i], wb + (i - L::NA) * 1024);
      } else if constexpr (i < L::NA + L::NCODE + L::NMETA) {
        pf_glds16(w.p1 + (L::Q6 ? kt * 16 : (kt >> 2) * 16) + off[i], wb + L::OFF_META);
      } else if constexpr (i < L::NA + L::NCODE + L::NMETA + L::NHB) {
        pf_glds16(w.p2 + (kt >> 2) * 32 + off[i], wb + L::OFF_HB);
      } else if constexpr (i < L::NA + L::NCODE + L::NMETA + L::NHB + L::NSC) {
        pf_glds4((L::Q6 ? w.p2 : w.p1) + kt * 4 + off[i], wb + L::OFF_SC);
      } else {
        pf_glds4(w.p3 + (((off[i] + (uint32_t)(kt >> 2)) >> 1) << 2), wb + L::OFF_DW);
      }
    });
  }
};

// raw B bytes of tile column cl (0..WC-1 of this wave) for lane half h
template <int QT, int BM, int WC>
__device__ __forceinline__ void pf4_braw(const uint8_t* wbase, int cl, int h, PfBRaw32& r) {
  using L = Pf4Layout<QT, BM, WC>;
  if constexpr (L::BF) {
    const uint8_t* row = wbase + cl * 128;
    const int x = (cl >> 1) & 7;
    r.mt = *(const uint4*)(row + (((0 + h) ^ x) << 4));
    r.b1 = *(const uint4*)(row + (((2 + h) ^ x) << 4));
    r.b2 = *(const uint4*)(row + (((4 + h) ^ x) << 4));
    r.b3 = *(const uint4*)(row + (((6 + h) ^ x) << 4));
  } else if constexpr (L::L8) {  // fragment s: bytes 16 s + 8 h .. of the column's 64
    const uint8_t* row = wbase + cl * 64 + 8 * h;
    r.c0 = *(const uint2*)(row);
    r.c1 = *(const uint2*)(row + 16);
    const uint2 c2 = *(const uint2*)(row + 32), c3 = *(const uint2*)(row + 48);
    r.b1 = make_uint4(c2.x, c2.y, c3.x, c3.y);
    r.scw = *(const uint32_t*)(wbase + L::OFF_SC + cl * 4);
  } else {
    r.c0 = *(const uint2*)(wbase + cl * 32 + 8 * h);
    r.c1 = *(const uint2*)(wbase + cl * 32 + 16 + 8 * h);
    if constexpr (L::META > 0) r.mt = *(const uint4*)(wbase + L::OFF_META + cl * 16);
    if constexpr (L::Q5) {  // qh bytes 8 h .. and 16 + 8 h .. of the block's 32
      const uint2 q0 = *(const uint2*)(wbase + L::OFF_HB + cl * 32 + 8 * h);
      const uint2 q1 = *(const uint2*)(wbase + L::OFF_HB + cl * 32 + 16 + 8 * h);
      r.b1 = make_uint4(q0.x, q0.y, q1.x, q1.y);
    }
    if constexpr (L::SC > 0) r.scw = *(const uint32_t*)(wbase + L::OFF_SC + cl * 4);
    if constexpr (L::Q6) r.dw = *(const uint32_t*)(wbase + L::OFF_DW + cl * 4);
  }
}

template <int QT, int BM, int WC, int EPI, int PROBE = 0>
__device__ __forceinline__ void pf4_body(const GemmQArgs& a, int m0, int n0, int seg, int kt0, int kt1, int S) {
  using L = Pf4Layout<QT, BM, WC>;
  constexpr int MT = BM / 32, CT = WC / 32, NS = L::NS, PW = L::PW;
  extern __shared__ __attribute__((aligned(16))) uint8_t pf_smem[];
  const int tid = threadIdx.x, lane = tid & 63;
  const int wv = __builtin_amdgcn_readfirstlane(tid >> 6);
  QWeight w;
  w.qtype = QT;
  w.rows = seg == 0 ? a.seg[0].rows : (seg == 1 ? a.seg[1].rows : a.seg[2].rows);
  w.cols = a.K;
  w.pad_ = 0;
  w.p0 = seg == 0 ? a.seg[0].p0 : (seg == 1 ? a.seg[1].p0 : a.seg[2].p0);
  w.p1 = seg == 0 ? a.seg[0].p1 : (seg == 1 ? a.seg[1].p1 : a.seg[2].p1);
  w.p2 = seg == 0 ? a.seg[0].p2 : (seg == 1 ? a.seg[1].p2 : a.seg[2].p2);
  w.p3 = seg == 0 ? a.seg[0].p3 : (seg == 1 ? a.seg[1].p3 : a.seg[2].p3);
  const int wcol0 = n0 - (seg == 0 ? a.seg_n0[0] : (seg == 1 ? a.seg_n0[1] : a.seg_n0[2])) + wv * WC;
  const uint32_t nbk = (uint32_t)a.K >> 8;
  const int r32 = lane & 31, h = lane >> 5;

  gf32x16 acc[MT][CT];
#pragma unroll
  for (int i = 0; i < MT; ++i)
#pragma unroll
    for (int c = 0; c < CT; ++c)
#pragma unroll
      for (int e = 0; e < 16; ++e) acc[i][c][e] = 0.f;

  const int nk = kt1 - kt0;
  Pf4Dma<QT, BM, WC> dma;
  const uint32_t lds0 = __builtin_amdgcn_readfirstlane(pf_lds_addr(pf_smem));
  dma.init(a, wcol0, m0, wv);
  // Pipeline: NS slots, all NS filled ahead.  The barrier B(t+1) sits inside step t's last phase,
  // between its two MFMA halves: by then every wave has waited for its own step-(t+1) pieces
  // (phase 1) and holds step t's last fragments in registers, so slot t is free for DMA(t + NS) and
  // step t+1's first A reads fly under the remaining MFMAs.  The loop is branch-free (a branch splits
  // the scheduling region and, here, made the allocator shuttle accumulators between AGPRs and
  // VGPRs): past the last step the DMA re-loads step nk-1 into the free slot and the decode reads a
  // stale slot, neither ever consumed; every DMA is drained before the epilogue.
  const int klast = kt1 - 1;
#pragma unroll
  for (int p = 0; p < NS; ++p) dma.template issue<PROBE>(a, w, min(kt0 + p, klast), lds0 + p * L::SLOT, wv);

  // B fragments: bf[c][s] is consumed by phase s; the next step's fragment s is decoded into it in
  // the phase after (s = 0..2 in phases 1..3 of this step, s = 3 in phase 0 of the next), from raw
  // bytes read once per column in phase 1 -- one fragment per column per phase, no second set.
  gbf16x8 bf[CT][4], fa[MT], fb[MT];
  PfBRaw32 raw[CT];
  int rkt = kt0;  // K-step of raw
  auto read_raw = [&](const uint8_t* sl, int kt) __attribute__((always_inline)) {
#pragma unroll
    for (int c = 0; c < CT; ++c) pf4_braw<QT, BM, WC>(sl + L::OFF_B + wv * L::WB, 32 * c + r32, h, raw[c]);
    rkt = kt;
  };
  auto dec = [&](auto sc) __attribute__((always_inline)) {
    constexpr int S4 = decltype(sc)::value;
#pragma unroll
    for (int c = 0; c < CT; ++c) {
      const int cl = 32 * c + r32;
      const int dpar = L::Q6 ? (int)(((uint32_t)(wcol0 + cl) * nbk + (uint32_t)(rkt >> 2)) & 1u) : 0;
      bf[c][S4] = pf_bdec32<QT, S4>(raw[c], h, rkt, dpar);
      // pinned here: LLVM otherwise sinks the arithmetic to its first use (the next step, past the
      // barrier), where it ran serially with the matrix pipe idle
      asm volatile("" : "+v"(bf[c][S4]));
    }
  };
  auto ldA = [&](const uint8_t* sl, gbf16x8(&f)[MT], int sp) __attribute__((always_inline)) {
#pragma unroll
    for (int i = 0; i < MT; ++i) {
      const int row = 32 * i + r32;
      const uint4 av = *(const uint4*)(sl + row * 128 + (((2 * sp + h) ^ ((row >> 1) & 7)) << 4));
      __builtin_memcpy(&f[i], &av, 16);
    }
  };
  auto mfma_range = [&](const gbf16x8(&f)[MT], int sp, int k0, int k1) __attribute__((always_inline)) {
#pragma unroll
    for (int k = 0; k < MT * CT; ++k) {
      if (k < k0 || k >= k1) continue;
      const int c = k / MT, i = k % MT;
      acc[i][c] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(f[i], bf[c][sp], acc[i][c], 0, 0, 0);
    }
  };
  constexpr int NMF = MT * CT, HALF = NMF / 2;
  // step kt0's own pieces (NS - 1 younger steps in flight)
  if constexpr (!(PROBE & 1)) {
    pf_vmcnt<(NS - 1) * PW>();
  }
  read_raw(pf_smem, kt0);
  dec(std::integral_constant<int, 0>{});
  dec(std::integral_constant<int, 1>{});
  dec(std::integral_constant<int, 2>{});
  asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
  pf_barrier();
  ldA(pf_smem, fa, 0);

  int cur = 0;
  for (int t = 0; t < nk; ++t) {
    const uint8_t* slot = pf_smem + cur * L::SLOT;
    const int nxt = cur == NS - 1 ? 0 : cur + 1;
    __builtin_amdgcn_sched_barrier(0);
    // phase 0: step t's fragment 3
    ldA(slot, fb, 1);
    dec(std::integral_constant<int, 3>{});
    mfma_range(fa, 0, 0, NMF);
    __builtin_amdgcn_sched_barrier(0);
    // phase 1: own step-(t+1) pieces landed (NS - 2 younger steps in flight) -> raw bytes, fragment 0
    ldA(slot, fa, 2);
    if constexpr (!(PROBE & 1)) {
      pf_vmcnt<(NS - 2) * PW>();
    }
    read_raw(pf_smem + nxt * L::SLOT, kt0 + t + 1);
    dec(std::integral_constant<int, 0>{});
    mfma_range(fb, 1, 0, NMF);
    __builtin_amdgcn_sched_barrier(0);
    // phase 2
    ldA(slot, fb, 3);
    dec(std::integral_constant<int, 1>{});
    mfma_range(fa, 2, 0, NMF);
    __builtin_amdgcn_sched_barrier(0);
    // phase 3: half the MFMAs; B(t+1); step t+1's first reads, DMA(t + NS) into slot t, fragment 2
    // of step t+1, under the other half
    mfma_range(fb, 3, 0, HALF);
    __builtin_amdgcn_sched_barrier(0);
    asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
    if constexpr (!(PROBE & 8)) pf_barrier();
    ldA(pf_smem + nxt * L::SLOT, fa, 0);
    if constexpr (!(PROBE & 4)) dma.template issue<PROBE>(a, w, min(kt0 + t + NS, klast), lds0 + cur * L::SLOT, wv);
    dec(std::integral_constant<int, 2>{});
    mfma_range(fb, 3, HALF, NMF);
    cur = nxt;
  }
  pf_vmcnt<0>();  // no LDS-DMA may land after this workgroup's LDS is released

  // epilogue -- C/D map of the 32x32 accumulator: col = lane & 31, row = (e & 3) + 8 (e >> 2) + 4 h
#pragma unroll
  for (int c = 0; c < CT; ++c) {
    const int n = n0 + wv * WC + 32 * c + r32;
#pragma unroll
    for (int i = 0; i < MT; ++i) {
#pragma unroll
      for (int e = 0; e < 16; ++e) {
        const int m = m0 + 32 * i + (e & 3) + 8 * (e >> 2) + 4 * h;
        const float v = acc[i][c][e];
        if constexpr (EPI == GEPI_SWIGLU_BF16) {
          const float up = __int_as_float(__builtin_amdgcn_mov_dpp(__float_as_int(v), 0xB1, 0xF, 0xF, false));
          if (m < a.M && !(r32 & 1)) a.C16[(size_t)m * a.ldc + (n >> 1)] = f32_to_bf16(glu_act(v, a.act) * up);
        } else if constexpr (EPI == GEPI_STORE16) {
          if (m < a.M) a.C16[(size_t)m * a.ldc + n] = f32_to_bf16(store16_val(a, n, v));
        } else if constexpr (EPI == GEPI_QKV) {
          pf_qkv_out(a, m, n, v, !(r32 & 1));
        } else if (m < a.M) {
          float* cp = a.C + (size_t)m * a.ldc + n;
          if (S > 1) unsafeAtomicAdd(cp, v);
          else if constexpr (EPI == GEPI_ACCUM) *cp += v;
          else *cp = v;
        }
      }
    }
  }
}

// ==== pf8: 8 waves (two per SIMD) x 32 columns, 16x16x32 MFMA ======================================
// The 8-wave 16x16x32 body ran the compute-only probe at 1.33 PF per busy CU against 1.16 for pf4's
// one wave per SIMD (the SIMD's second wave covers the first's LDS latencies); this is that body
// with pf4's structure: compile-time own-column DMA pieces, the next step's B decode inside this
// step's phases, the barrier between the two halves of the last phase, a branch-free loop.
template <int QT, int BM, int EPI, int PROBE = 0>
__device__ __forceinline__ void pf8_body(const GemmQArgs& a, int m0, int n0, int seg, int kt0, int kt1, int S) {
  constexpr int NW = 8, WC = 32;
  using L = Pf4Layout<QT, BM, WC, NW>;
  constexpr int MT = BM / 16, GR = MT < 8 ? MT : 8, NG = MT / GR, NPH = 2 * NG, NS = L::NS, PW = L::PW;
  extern __shared__ __attribute__((aligned(16))) uint8_t pf_smem[];
  const int tid = threadIdx.x, lane = tid & 63;
  const int wv = __builtin_amdgcn_readfirstlane(tid >> 6);
  QWeight w;
  w.qtype = QT;
  w.rows = seg == 0 ? a.seg[0].rows : (seg == 1 ? a.seg[1].rows : a.seg[2].rows);
  w.cols = a.K;
  w.pad_ = 0;
  w.p0 = seg == 0 ? a.seg[0].p0 : (seg == 1 ? a.seg[1].p0 : a.seg[2].p0);
  w.p1 = seg == 0 ? a.seg[0].p1 : (seg == 1 ? a.seg[1].p1 : a.seg[2].p1);
  w.p2 = seg == 0 ? a.seg[0].p2 : (seg == 1 ? a.seg[1].p2 : a.seg[2].p2);
  w.p3 = seg == 0 ? a.seg[0].p3 : (seg == 1 ? a.seg[1].p3 : a.seg[2].p3);
  const int wcol0 = n0 - (seg == 0 ? a.seg_n0[0] : (seg == 1 ? a.seg_n0[1] : a.seg_n0[2])) + wv * WC;
  const uint32_t nbk = (uint32_t)a.K >> 8;
  const int r16 = lane & 15, q = lane >> 4;

  gf32x4 acc[MT][2];
#pragma unroll
  for (int i = 0; i < MT; ++i)
#pragma unroll
    for (int c = 0; c < 2; ++c) acc[i][c] = gf32x4{0.f, 0.f, 0.f, 0.f};

  const int nk = kt1 - kt0, klast = kt1 - 1;
  Pf4Dma<QT, BM, WC, NW> dma;
  const uint32_t lds0 = __builtin_amdgcn_readfirstlane(pf_lds_addr(pf_smem));
  dma.init(a, wcol0, m0, wv);
#pragma unroll
  for (int p = 0; p < NS; ++p) dma.template issue<PROBE>(a, w, min(kt0 + p, klast), lds0 + p * L::SLOT, wv);

  gbf16x8 bf[2][2], fa[GR], fb[GR];
  PfBRaw raw[2];
  int rkt = kt0;
  auto read_raw = [&](const uint8_t* sl, int kt) __attribute__((always_inline)) {
    const uint8_t* wb = sl + L::OFF_B + wv * L::WB;
#pragma unroll
    for (int c = 0; c < 2; ++c) {
      const int cl = 16 * c + r16;
      PfBRaw& r = raw[c];
      if constexpr (L::BF) {
        r.mt = *(const uint4*)(wb + cl * 128 + (((0 + q) ^ ((cl >> 1) & 7)) << 4));
        r.b1 = *(const uint4*)(wb + cl * 128 + (((4 + q) ^ ((cl >> 1) & 7)) << 4));
      } else if constexpr (L::L8 || L::L0) {  // the K-step's two 32-blocks: bytes of fragment 0 / 1
        const int bs = L::L8 ? 32 : 16, o = L::L8 ? 8 * q : 8 * (q & 1);
        r.cw = *(const uint2*)(wb + cl * (2 * bs) + o);
        const uint2 c1 = *(const uint2*)(wb + cl * (2 * bs) + bs + o);
        r.b1.x = c1.x;
        r.b1.y = c1.y;
        r.scw = *(const uint32_t*)(wb + L::OFF_SC + cl * 4);
      } else {
        r.cw = *(const uint2*)(wb + cl * 32 + 8 * q);
        if constexpr (L::Q5) r.hb = *(const uint2*)(wb + L::OFF_HB + cl * 32 + 8 * q);
        if constexpr (L::Q6) {
          r.hb = *(const uint2*)(wb + L::CODE + cl * 16 + 8 * (q >> 1));
          r.scw = *(const uint32_t*)(wb + L::CODE + L::META + cl * 4);
          r.dw = *(const uint32_t*)(wb + L::OFF_DW + cl * 4);
        } else {
          r.mt = *(const uint4*)(wb + L::OFF_META + cl * 16);
        }
      }
    }
    rkt = kt;
  };
  auto dec = [&](auto sc) __attribute__((always_inline)) {
    constexpr int S2 = decltype(sc)::value;
#pragma unroll
    for (int c = 0; c < 2; ++c) {
      const int cl = 16 * c + r16;
      const int dpar = L::Q6 ? (int)(((uint32_t)(wcol0 + cl) * nbk + (uint32_t)(rkt >> 2)) & 1u) : 0;
      bf[c][S2] = pf_bdec<QT, S2>(raw[c], q, rkt, dpar);
      asm volatile("" : "+v"(bf[c][S2]));  // keep the decode in this phase (else sunk past the barrier)
    }
  };
  auto ldA = [&](const uint8_t* sl, gbf16x8(&f)[GR], int p) __attribute__((always_inline)) {
    const int sp = p / NG, g = p % NG;
#pragma unroll
    for (int i = 0; i < GR; ++i) {
      const int row = 16 * (g * GR + i) + r16;
      const uint4 av = *(const uint4*)(sl + row * 128 + (((4 * sp + q) ^ ((row >> 1) & 7)) << 4));
      __builtin_memcpy(&f[i], &av, 16);
    }
  };
  auto mfma_range = [&](const gbf16x8(&f)[GR], int p, int k0, int k1) __attribute__((always_inline)) {
    const int sp = p / NG, g = p % NG;
#pragma unroll
    for (int k = 0; k < 2 * GR; ++k) {
      if (k < k0 || k >= k1) continue;
      const int c = k / GR, i = k % GR;
      acc[g * GR + i][c] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(f[i], bf[c][sp], acc[g * GR + i][c], 0, 0, 0);
    }
  };
  if constexpr (!(PROBE & 1)) {
    pf_vmcnt<(NS - 1) * PW>();
  }
  read_raw(pf_smem, kt0);
  dec(std::integral_constant<int, 0>{});
  asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
  pf_barrier();
  ldA(pf_smem, fa, 0);

  int cur = 0;
  for (int t = 0; t < nk; ++t) {
    const uint8_t* slot = pf_smem + cur * L::SLOT;
    const int nxt = cur == NS - 1 ? 0 : cur + 1;
    static_for<NPH>([&](auto pc) {
      constexpr int p = decltype(pc)::value;
      __builtin_amdgcn_sched_barrier(0);
      auto& cf = (p % 2 == 0) ? fa : fb;
      auto& nf = (p % 2 == 0) ? fb : fa;
      if constexpr (p + 1 < NPH) ldA(slot, nf, p + 1);
      if constexpr (p == 0) dec(std::integral_constant<int, 1>{});  // this step's fragment 1
      if constexpr (p == NG) {
        // own pieces of step t+1 landed (NS - 2 younger steps in flight): its raw bytes, fragment 0
        if constexpr (!(PROBE & 1)) {
          pf_vmcnt<(NS - 2) * PW>();
        }
        read_raw(pf_smem + nxt * L::SLOT, kt0 + t + 1);
        dec(std::integral_constant<int, 0>{});
      }
      if constexpr (p + 1 < NPH) {
        mfma_range(cf, p, 0, 2 * GR);
      } else {
        // last phase: half the MFMAs; B(t+1); the next step's first reads and DMA(t + NS) into slot t
        // under the other half
        mfma_range(cf, p, 0, GR);
        __builtin_amdgcn_sched_barrier(0);
        asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
        if constexpr (!(PROBE & 8)) pf_barrier();
        ldA(pf_smem + nxt * L::SLOT, nf, 0);
        if constexpr (!(PROBE & 4)) dma.template issue<PROBE>(a, w, min(kt0 + t + NS, klast), lds0 + cur * L::SLOT, wv);
        mfma_range(cf, p, GR, 2 * GR);
      }
    });
    if constexpr (NPH % 2 == 1) {
#pragma unroll
      for (int i = 0; i < GR; ++i) fa[i] = fb[i];
    }
    cur = nxt;
  }
  pf_vmcnt<0>();  // no LDS-DMA may land after this workgroup's LDS is released

  // epilogue -- C/D map of the 16x16 accumulator: col = lane & 15, row = 4 * (lane >> 4) + e
#pragma unroll
  for (int c = 0; c < 2; ++c) {
    const int n = n0 + wv * WC + 16 * c + r16;
#pragma unroll
    for (int i = 0; i < MT; ++i) {
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const int m = m0 + 16 * i + 4 * q + e;
        const float v = acc[i][c][e];
        if constexpr (EPI == GEPI_SWIGLU_BF16) {
          const float up = __int_as_float(__builtin_amdgcn_mov_dpp(__float_as_int(v), 0xB1, 0xF, 0xF, false));
          if (m < a.M && !(r16 & 1)) a.C16[(size_t)m * a.ldc + (n >> 1)] = f32_to_bf16(glu_act(v, a.act) * up);
        } else if constexpr (EPI == GEPI_STORE16) {
          if (m < a.M) a.C16[(size_t)m * a.ldc + n] = f32_to_bf16(store16_val(a, n, v));
        } else if constexpr (EPI == GEPI_QKV) {
          pf_qkv_out(a, m, n, v, !(r16 & 1));
        } else if (m < a.M) {
          float* cp = a.C + (size_t)m * a.ldc + n;
          if (S > 1) unsafeAtomicAdd(cp, v);
          else if constexpr (EPI == GEPI_ACCUM) *cp += v;
          else *cp = v;
        }
      }
    }
  }
}

// ==== pf8c: pf8 with the K-quant weight planes staged coalesced ==================================
// Round-5 probe (bench_gemm.py --pf-probe 216/316): the per-step weight pieces -- each column's 32 B
// of codes and its 16-B scale record, i.e. 32-64 separate rows per DMA instruction -- cost 13-18 %
// of the kernel against contiguous pieces.  Here a wave stages, per HALF block (2 K-steps), 64
// contiguous bytes of codes per column (16 rows x 64 B per DMA: 4 lanes per row, the 16-B units
// XOR-swizzled by (row >> 2) & 3 on the source side so the 8-byte fragment reads are conflict-free),
// per 256-block the scale records (Q4_K meta / Q6_K int8 scales: 16 B per row) and Q6_K d, and the
// Q6_K high bits per half block (32 B per row); double buffers by half-block / block parity.
// Every step issues the same group (so one vmcnt immediate): the per-block / per-half-block planes
// go as partial-lane pieces, one per step (records: 8 rows = 32 lanes x 4 B; Q6_K d: 8 lanes).
// Group G(s), issued at the end of step s (after the barrier B(s+1)), s relative to the slice:
//   A(s + 3); code piece (s & 1) [+ Q6_K high-bit piece (s & 1)] of half block (s + 4) / 2;
//   record piece (s + 6) % 4 [+ Q6_K d piece] of block (s + 6) / 4.
// Every target buffer is free by then (its previous contents were last decoded during step s); the
// data is needed by the decode of the first step using it, at least 1.25 steps later.
template <int QT, int BM>
struct PfcLayout {
  static constexpr int NW = 8, WC = 32, NSA = 3;
  static constexpr bool Q6 = QT == QT_Q6_K;
  static constexpr int A_BYTES = BM * 128;
  static constexpr int OFF_CB = NSA * A_BYTES, CB_W = WC * 64;
  static constexpr int OFF_HB = OFF_CB + 2 * NW * CB_W, HB_W = Q6 ? WC * 32 : 0;  // Q6_K high bits
  static constexpr int OFF_RB = OFF_HB + 2 * NW * HB_W, RB_W = WC * 16;           // records
  static constexpr int OFF_D = OFF_RB + 2 * NW * RB_W, D_W = Q6 ? WC * 4 : 0;
  static constexpr int TOTAL = OFF_D + 2 * NW * D_W;
  static constexpr int NA = BM / 64;
  static constexpr int PW = NA + 2 + (Q6 ? 2 : 0);     // DMA instructions per wave per step
  static constexpr int PRE = NA + 6 + (Q6 ? 6 : 0);    // prologue group: step 0's A, half block 0, block 0
};

template <int QT, int BM>
struct PfcDma {
  using L = PfcLayout<QT, BM>;
  static constexpr int NW = 8;
  uint32_t offA[L::NA], offC[2], offR, offH, offD;

  __device__ __forceinline__ void init(const GemmQArgs& a, int wcol0, int m0, int wv) {
    const int lane = threadIdx.x & 63;
    const uint32_t nbk = (uint32_t)a.K >> 8;
#pragma unroll
    for (int i = 0; i < L::NA; ++i) {
      const int p = 64 * (NW * i + wv) + lane, row = p >> 3, c = (p & 7) ^ ((row >> 1) & 7);
      const int m = min(m0 + row, a.M - 1);
      offA[i] = ((uint32_t)m * (uint32_t)a.lda + (uint32_t)(c * 8)) * 2u;
    }
#pragma unroll
    for (int pc = 0; pc < 2; ++pc) {
      const int row = 16 * pc + (lane >> 2), u = (lane & 3) ^ ((row >> 2) & 3);
      offC[pc] = (uint32_t)(wcol0 + row) * nbk * 128u + 16u * (uint32_t)u;
    }
    const int l32 = lane & 31;
    offR = (uint32_t)(wcol0 + (l32 >> 2)) * nbk * 16u + 4u * (uint32_t)(l32 & 3);  // + 8 rows per piece
    offH = (uint32_t)(wcol0 + (l32 >> 1)) * nbk * 64u + 16u * (uint32_t)(l32 & 1);  // + 16 rows per piece
    offD = (uint32_t)(wcol0 + (lane & 7)) * nbk;                                      // + 8 rows per piece
  }

  __device__ __forceinline__ void A(const GemmQArgs& a, int kt, uint32_t dst, int wv) const {
#pragma unroll
    for (int i = 0; i < L::NA; ++i) pf_glds16((const uint8_t*)a.A + kt * 128 + offA[i], dst + (NW * i + wv) * 1024);
  }
  // the A pieces i with i % NP == P
  template <int P, int NP>
  __device__ __forceinline__ void A_part(const GemmQArgs& a, int kt, uint32_t dst, int wv) const {
#pragma unroll
    for (int i = 0; i < L::NA; ++i)
      if (i % NP == P) pf_glds16((const uint8_t*)a.A + kt * 128 + offA[i], dst + (NW * i + wv) * 1024);
  }
  // code piece pc of half block hsrc into the wave's half-block buffer at dst
  __device__ __forceinline__ void code(const QWeight& w, int hsrc, int pc, uint32_t dst) const {
    // (a register select: offC[pc] with a runtime pc puts the array in scratch, and the scratch
    // load's vmcnt(0) drained every in-flight DMA)
    pf_glds16(w.p0 + hsrc * 64 + (pc ? offC[1] : offC[0]), dst + pc * 1024);
  }
  // record piece pr (rows 8 pr .. 8 pr + 7) of block bsrc; lanes 0..31
  __device__ __forceinline__ void rec(const QWeight& w, int bsrc, int pr, uint32_t nbk, uint32_t dst) const {
    if ((threadIdx.x & 63) < 32) pf_glds4((L::Q6 ? w.p2 : w.p1) + bsrc * 16 + offR + pr * 128 * nbk, dst + pr * 128);
  }
  // Q6_K high-bit piece pc (rows 16 pc ..) of half block hsrc; lanes 0..31
  __device__ __forceinline__ void hi(const QWeight& w, int hsrc, int pc, uint32_t nbk, uint32_t dst) const {
    if ((threadIdx.x & 63) < 32) pf_glds16(w.p1 + hsrc * 32 + offH + pc * 1024 * nbk, dst + pc * 512);
  }
  // Q6_K d piece pr (rows 8 pr ..) of block bsrc: the dword holding each row's f16 d; lanes 0..7
  __device__ __forceinline__ void dq(const QWeight& w, int bsrc, int pr, uint32_t nbk, uint32_t dst) const {
    if ((threadIdx.x & 63) < 8) pf_glds4(w.p3 + (((offD + pr * 8 * nbk + (uint32_t)bsrc) * 2u) & ~3u), dst + pr * 32);
  }
};

template <int QT, int BM, int EPI, int PROBE = 0>
__device__ __forceinline__ void pf8c_body(const GemmQArgs& a, int m0, int n0, int seg, int kt0, int kt1, int S) {
  using L = PfcLayout<QT, BM>;
  constexpr int NW = 8, WC = 32, NSA = L::NSA, PW = L::PW;
  // row tiles per phase: 4 at BM = 256 (8 phases; 8 ran out of registers once the DMA is spread)
  constexpr int MT = BM / 16, GR = MT >= 16 ? 4 : MT, NG = MT / GR, NPH = 2 * NG;
  extern __shared__ __attribute__((aligned(16))) uint8_t pf_smem[];
  const int tid = threadIdx.x, lane = tid & 63;
  const int wv = __builtin_amdgcn_readfirstlane(tid >> 6);
  QWeight w;
  w.qtype = QT;
  w.rows = seg == 0 ? a.seg[0].rows : (seg == 1 ? a.seg[1].rows : a.seg[2].rows);
  w.cols = a.K;
  w.pad_ = 0;
  w.p0 = seg == 0 ? a.seg[0].p0 : (seg == 1 ? a.seg[1].p0 : a.seg[2].p0);
  w.p1 = seg == 0 ? a.seg[0].p1 : (seg == 1 ? a.seg[1].p1 : a.seg[2].p1);
  w.p2 = seg == 0 ? a.seg[0].p2 : (seg == 1 ? a.seg[1].p2 : a.seg[2].p2);
  w.p3 = seg == 0 ? a.seg[0].p3 : (seg == 1 ? a.seg[1].p3 : a.seg[2].p3);
  const int wcol0 = n0 - (seg == 0 ? a.seg_n0[0] : (seg == 1 ? a.seg_n0[1] : a.seg_n0[2])) + wv * WC;
  const uint32_t nbk = (uint32_t)a.K >> 8;
  const int r16 = lane & 15, q = lane >> 4;

  gf32x4 acc[MT][2];
#pragma unroll
  for (int i = 0; i < MT; ++i)
#pragma unroll
    for (int c = 0; c < 2; ++c) acc[i][c] = gf32x4{0.f, 0.f, 0.f, 0.f};

  // kt0, kt1 are multiples of 4 (block-aligned slices)
  const int nk = kt1 - kt0, klast = kt1 - 1, hlast = (kt1 >> 1) - 1, blast = (kt1 >> 2) - 1;
  PfcDma<QT, BM> dma;
  const uint32_t lds0 = __builtin_amdgcn_readfirstlane(pf_lds_addr(pf_smem));
  dma.init(a, wcol0, m0, wv);
  constexpr uint32_t CBS = NW * L::CB_W, HBS = NW * L::HB_W, RBS = NW * L::RB_W, DBS = NW * L::D_W;
  const uint32_t cb = lds0 + L::OFF_CB + wv * L::CB_W, hb = lds0 + L::OFF_HB + wv * L::HB_W;
  const uint32_t rb = lds0 + L::OFF_RB + wv * L::RB_W, db = lds0 + L::OFF_D + wv * L::D_W;
  // G(s): phase-split -- A pieces in the first phases (longest lead), then code (+ high bits), then
  // records (+ d); PH_ALL = every phase (prologue)
  constexpr int PH_ALL = -1;
  auto group = [&](int s, auto phc) __attribute__((always_inline)) {
    constexpr int ph = decltype(phc)::value;
    // A piece i in phase i % NG (all before the decode wait at phase NG)
    if constexpr (ph == PH_ALL) {
      dma.A(a, min(kt0 + s + NSA, klast), lds0 + (uint32_t)(((s + 3 * NSA) % NSA) * L::A_BYTES), wv);
    } else if constexpr (ph < NG) {
      dma.template A_part<(ph < 0 ? 0 : ph), NG>(a, min(kt0 + s + NSA, klast),
                                                 lds0 + (uint32_t)(((s + 3 * NSA) % NSA) * L::A_BYTES), wv);
    }
    const int H = (kt0 >> 1) + ((s + 4) >> 1), B = (kt0 >> 2) + ((s + 6) >> 2), pr = (s + 6) & 3;
    if constexpr (ph == PH_ALL || ph == NPH - 2 || (NPH == 2 && ph == 0)) {
      dma.code(w, min(H, hlast), s & 1, cb + (uint32_t)(H & 1) * CBS);
      if constexpr (L::Q6) dma.hi(w, min(H, hlast), s & 1, nbk, hb + (uint32_t)(H & 1) * HBS);
    }
    if constexpr (ph == PH_ALL || ph == NPH - 1) {
      dma.rec(w, min(B, blast), pr, nbk, rb + (uint32_t)(B & 1) * RBS);
      if constexpr (L::Q6) dma.dq(w, min(B, blast), pr, nbk, db + (uint32_t)(B & 1) * DBS);
    }
  };
  // DMA instructions of G(s-1) issued in step s's phases before the decode wait (phase NG)
  constexpr int NB = 1 + (L::Q6 ? 1 : 0);  // code pieces (+ high bits)
  constexpr int PRE_WAIT = NPH == 2 ? L::NA + NB : L::NA;
  {  // prologue: step 0's A, half block 0, block 0 (PRE instructions), then G(-2), G(-1)
    const int H0 = kt0 >> 1, B0 = kt0 >> 2;
    dma.A(a, kt0, lds0, wv);
    dma.code(w, H0, 0, cb + (uint32_t)(H0 & 1) * CBS);
    dma.code(w, H0, 1, cb + (uint32_t)(H0 & 1) * CBS);
    if constexpr (L::Q6) {
      dma.hi(w, H0, 0, nbk, hb + (uint32_t)(H0 & 1) * HBS);
      dma.hi(w, H0, 1, nbk, hb + (uint32_t)(H0 & 1) * HBS);
    }
#pragma unroll
    for (int pr = 0; pr < 4; ++pr) {
      dma.rec(w, B0, pr, nbk, rb + (uint32_t)(B0 & 1) * RBS);
      if constexpr (L::Q6) dma.dq(w, B0, pr, nbk, db + (uint32_t)(B0 & 1) * DBS);
    }
    group(-2, std::integral_constant<int, PH_ALL>{});
  }

  gbf16x8 bf[2][2], fa[GR], fb[GR];
  PfBRaw raw[2];
  int rkt = kt0;
  // raw bytes of (absolute) K-step kt for this lane's two columns
  auto read_raw = [&](int kt) __attribute__((always_inline)) {
    const int H = kt >> 1, j = kt & 1, B = kt >> 2;
    const uint8_t* cbp = pf_smem + L::OFF_CB + (H & 1) * CBS + wv * L::CB_W;
    const uint8_t* rbp = pf_smem + L::OFF_RB + (B & 1) * RBS + wv * L::RB_W;
#pragma unroll
    for (int c = 0; c < 2; ++c) {
      const int row = 16 * c + r16;
      PfBRaw& r = raw[c];
      r.cw = *(const uint2*)(cbp + row * 64 + (((2 * j + (q >> 1)) ^ ((row >> 2) & 3)) << 4) + 8 * (q & 1));
      if constexpr (L::Q6) {
        r.hb = *(const uint2*)(pf_smem + L::OFF_HB + (H & 1) * HBS + wv * L::HB_W + row * 32 + (2 * j + (q >> 1)) * 8);
        r.scw = *(const uint32_t*)(rbp + row * 16 + 4 * (kt & 3));
        r.dw = *(const uint32_t*)(pf_smem + L::OFF_D + (B & 1) * DBS + wv * L::D_W + row * 4);
      } else {
        r.mt = *(const uint4*)(rbp + row * 16);
      }
    }
    rkt = kt;
  };
  auto dec = [&](auto sc) __attribute__((always_inline)) {
    constexpr int S2 = decltype(sc)::value;
#pragma unroll
    for (int c = 0; c < 2; ++c) {
      const int cl = 16 * c + r16;
      const int dpar = L::Q6 ? (int)(((uint32_t)(wcol0 + cl) * nbk + (uint32_t)(rkt >> 2)) & 1u) : 0;
      bf[c][S2] = pf_bdec<QT, S2>(raw[c], q, rkt, dpar);
      asm volatile("" : "+v"(bf[c][S2]));  // keep the decode in this phase (else sunk past the barrier)
    }
  };
  auto ldA = [&](const uint8_t* sl, gbf16x8(&f)[GR], int p) __attribute__((always_inline)) {
    const int sp = p / NG, g = p % NG;
#pragma unroll
    for (int i = 0; i < GR; ++i) {
      const int row = 16 * (g * GR + i) + r16;
      const uint4 av = *(const uint4*)(sl + row * 128 + (((4 * sp + q) ^ ((row >> 1) & 7)) << 4));
      __builtin_memcpy(&f[i], &av, 16);
    }
  };
  auto mfma_range = [&](const gbf16x8(&f)[GR], int p, int k0, int k1) __attribute__((always_inline)) {
    const int sp = p / NG, g = p % NG;
#pragma unroll
    for (int k = 0; k < 2 * GR; ++k) {
      if (k < k0 || k >= k1) continue;
      const int c = k / GR, i = k % GR;
      acc[g * GR + i][c] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(f[i], bf[c][sp], acc[g * GR + i][c], 0, 0, 0);
    }
  };
  if constexpr (!(PROBE & 1)) pf_vmcnt<PW>();  // the prologue group landed (G(-2) in flight)
  read_raw(kt0);
  dec(std::integral_constant<int, 0>{});
  asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
  pf_barrier();
  ldA(pf_smem, fa, 0);

  int cur = 0;
  for (int s = 0; s < nk; ++s) {
    const uint8_t* slot = pf_smem + cur * L::A_BYTES;
    const int nxt = cur == NSA - 1 ? 0 : cur + 1;
    static_for<NPH>([&](auto pc) {
      constexpr int p = decltype(pc)::value;
      __builtin_amdgcn_sched_barrier(0);
      auto& cf = (p % 2 == 0) ? fa : fb;
      auto& nf = (p % 2 == 0) ? fb : fa;
      if constexpr (p + 1 < NPH) ldA(slot, nf, p + 1);
      if constexpr (p == 0) dec(std::integral_constant<int, 1>{});
      if constexpr (p == NG) {
        // G(s-2) landed -- step s+1's codes / records and this wave's A pieces of it -- with only
        // G(s-1)'s first-phase pieces younger
        if constexpr (!(PROBE & 1)) pf_vmcnt<PRE_WAIT>();
        read_raw(kt0 + s + 1);  // (past the last step: stale buffers, unused)
        dec(std::integral_constant<int, 0>{});
      }
      // G(s-1): its slot / buffers were released by B(s) (past the end: clamped re-loads, unused)
      if constexpr (!(PROBE & 4)) group(s - 1, pc);
      if constexpr (p + 1 < NPH) {
        mfma_range(cf, p, 0, 2 * GR);
      } else {
        mfma_range(cf, p, 0, GR);
        __builtin_amdgcn_sched_barrier(0);
        asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
        if constexpr (!(PROBE & 8)) pf_barrier();
        ldA(pf_smem + nxt * L::A_BYTES, nf, 0);
        mfma_range(cf, p, GR, 2 * GR);
      }
    });
    if constexpr (NPH % 2 == 1) {
#pragma unroll
      for (int i = 0; i < GR; ++i) fa[i] = fb[i];
    }
    cur = nxt;
  }
  pf_vmcnt<0>();  // no LDS-DMA may land after this workgroup's LDS is released

#pragma unroll
  for (int c = 0; c < 2; ++c) {
    const int n = n0 + wv * WC + 16 * c + r16;
#pragma unroll
    for (int i = 0; i < MT; ++i) {
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const int m = m0 + 16 * i + 4 * q + e;
        const float v = acc[i][c][e];
        if constexpr (EPI == GEPI_SWIGLU_BF16) {
          const float up = __int_as_float(__builtin_amdgcn_mov_dpp(__float_as_int(v), 0xB1, 0xF, 0xF, false));
          if (m < a.M && !(r16 & 1)) a.C16[(size_t)m * a.ldc + (n >> 1)] = f32_to_bf16(glu_act(v, a.act) * up);
        } else if constexpr (EPI == GEPI_STORE16) {
          if (m < a.M) a.C16[(size_t)m * a.ldc + n] = f32_to_bf16(store16_val(a, n, v));
        } else if constexpr (EPI == GEPI_QKV) {
          pf_qkv_out(a, m, n, v, !(r16 & 1));
        } else if (m < a.M) {
          float* cp = a.C + (size_t)m * a.ldc + n;
          if (S > 1) unsafeAtomicAdd(cp, v);
          else if constexpr (EPI == GEPI_ACCUM) *cp += v;
          else *cp = v;
        }
      }
    }
  }
}

// ==== pf8d: pf8c on v_mfma_f32_32x32x16_bf16 ======================================================
// PMC (round 5, gate/up M = 2048): with the DMA on, the waves spend +25 % active-instruction cycles
// (LDS-DMA issue ~55-60 cycles each) and the SIMD's issue port -- MFMA issue + decode VALU + DMA +
// LDS reads -- exceeds the matrix pipe's 2048 cycles per step.  A 32x32x16 MFMA holds vector issue
// for 8 of its 32 cycles against 8 of 16 for 16x16x32: half the MFMA issue cost at equal FLOPs.
// Wave tile BM rows x 32 columns = BM/32 accumulators; per K-step four k16 substeps (k = 16 s + 8 h
// + j: chunk (s & 1) bytes 8h.., low nibbles for s < 2).  Phase s uses fragment s; the next step's
// fragment s is decoded in phase s+1 (fragment 3 in the next step's phase 0) from raw bytes read
// after the phase-1 wait.  The staging is pf8c's (same layout, same DMA groups).
template <int QT, int BM, int EPI, int PROBE = 0>
__device__ __forceinline__ void pf8d_body(const GemmQArgs& a, int m0, int n0, int seg, int kt0, int kt1, int S) {
  using L = PfcLayout<QT, BM>;
  constexpr int NW = 8, WC = 32, NSA = L::NSA, PW = L::PW;
  // GD row tiles per phase (4 at BM = 256: two 8-fragment A buffers spill), ND phases per substep
  constexpr int MT = BM / 32, GD = MT > 4 ? 4 : MT, ND = MT / GD, NPH = 4 * ND;
  extern __shared__ __attribute__((aligned(16))) uint8_t pf_smem[];
  const int tid = threadIdx.x, lane = tid & 63;
  const int wv = __builtin_amdgcn_readfirstlane(tid >> 6);
  QWeight w;
  w.qtype = QT;
  w.rows = seg == 0 ? a.seg[0].rows : (seg == 1 ? a.seg[1].rows : a.seg[2].rows);
  w.cols = a.K;
  w.pad_ = 0;
  w.p0 = seg == 0 ? a.seg[0].p0 : (seg == 1 ? a.seg[1].p0 : a.seg[2].p0);
  w.p1 = seg == 0 ? a.seg[0].p1 : (seg == 1 ? a.seg[1].p1 : a.seg[2].p1);
  w.p2 = seg == 0 ? a.seg[0].p2 : (seg == 1 ? a.seg[1].p2 : a.seg[2].p2);
  w.p3 = seg == 0 ? a.seg[0].p3 : (seg == 1 ? a.seg[1].p3 : a.seg[2].p3);
  const int wcol0 = n0 - (seg == 0 ? a.seg_n0[0] : (seg == 1 ? a.seg_n0[1] : a.seg_n0[2])) + wv * WC;
  const uint32_t nbk = (uint32_t)a.K >> 8;
  const int r32 = lane & 31, h = lane >> 5;

  gf32x16 acc[MT];
#pragma unroll
  for (int i = 0; i < MT; ++i)
#pragma unroll
    for (int e = 0; e < 16; ++e) acc[i][e] = 0.f;

  const int nk = kt1 - kt0, klast = kt1 - 1, hlast = (kt1 >> 1) - 1, blast = (kt1 >> 2) - 1;
  PfcDma<QT, BM> dma;
  const uint32_t lds0 = __builtin_amdgcn_readfirstlane(pf_lds_addr(pf_smem));
  dma.init(a, wcol0, m0, wv);
  constexpr uint32_t CBS = NW * L::CB_W, HBS = NW * L::HB_W, RBS = NW * L::RB_W, DBS = NW * L::D_W;
  const uint32_t cb = lds0 + L::OFF_CB + wv * L::CB_W, hb = lds0 + L::OFF_HB + wv * L::HB_W;
  const uint32_t rb = lds0 + L::OFF_RB + wv * L::RB_W, db = lds0 + L::OFF_D + wv * L::D_W;
  // G(s) during step s+1, after the wait at phase ND: A pieces over phases ND .. ND + NAP - 1, code
  // (+ high bits) and records (+ d) in phase NPH - 2 (NPH - 1 at ND == 1); PH_ALL = every piece (prologue)
  constexpr int PH_ALL = -1, NAP = ND == 1 ? 2 : 4, PB = ND == 1 ? 3 : NPH - 2;
  auto group = [&](int s, auto phc) __attribute__((always_inline)) {
    constexpr int ph = decltype(phc)::value;
    const uint32_t adst = lds0 + (uint32_t)(((s + 3 * NSA) % NSA) * L::A_BYTES);
    const int ka = min(kt0 + s + NSA, klast);
    if constexpr (ph == PH_ALL) dma.A(a, ka, adst, wv);
    else if constexpr (ph >= ND && ph < ND + NAP) dma.template A_part<(ph - ND), NAP>(a, ka, adst, wv);
    const int H = (kt0 >> 1) + ((s + 4) >> 1), B = (kt0 >> 2) + ((s + 6) >> 2), pr = (s + 6) & 3;
    if constexpr (ph == PH_ALL || ph == PB) {
      dma.code(w, min(H, hlast), s & 1, cb + (uint32_t)(H & 1) * CBS);
      if constexpr (L::Q6) dma.hi(w, min(H, hlast), s & 1, nbk, hb + (uint32_t)(H & 1) * HBS);
      dma.rec(w, min(B, blast), pr, nbk, rb + (uint32_t)(B & 1) * RBS);
      if constexpr (L::Q6) dma.dq(w, min(B, blast), pr, nbk, db + (uint32_t)(B & 1) * DBS);
    }
  };
  {  // prologue: step 0's A, half block 0, block 0, then G(-2)
    const int H0 = kt0 >> 1, B0 = kt0 >> 2;
    dma.A(a, kt0, lds0, wv);
    dma.code(w, H0, 0, cb + (uint32_t)(H0 & 1) * CBS);
    dma.code(w, H0, 1, cb + (uint32_t)(H0 & 1) * CBS);
    if constexpr (L::Q6) {
      dma.hi(w, H0, 0, nbk, hb + (uint32_t)(H0 & 1) * HBS);
      dma.hi(w, H0, 1, nbk, hb + (uint32_t)(H0 & 1) * HBS);
    }
#pragma unroll
    for (int pr = 0; pr < 4; ++pr) {
      dma.rec(w, B0, pr, nbk, rb + (uint32_t)(B0 & 1) * RBS);
      if constexpr (L::Q6) dma.dq(w, B0, pr, nbk, db + (uint32_t)(B0 & 1) * DBS);
    }
    group(-2, std::integral_constant<int, PH_ALL>{});
  }

  gbf16x8 bf[4], fa[GD], fb[GD];
  PfBRaw32 raw;
  int rkt = kt0;
  auto read_raw = [&](int kt) __attribute__((always_inline)) {
    const int H = kt >> 1, j = kt & 1, B = kt >> 2;
    const uint8_t* cbp = pf_smem + L::OFF_CB + (H & 1) * CBS + wv * L::CB_W + r32 * 64;
    const uint8_t* rbp = pf_smem + L::OFF_RB + (B & 1) * RBS + wv * L::RB_W + r32 * 16;
    const int x = (r32 >> 2) & 3;
    raw.c0 = *(const uint2*)(cbp + (((2 * j) ^ x) << 4) + 8 * h);
    raw.c1 = *(const uint2*)(cbp + (((2 * j + 1) ^ x) << 4) + 8 * h);
    if constexpr (L::Q6) {
      // high bits {c0 run0, c0 run1, c1 run0, c1 run1} of this step's two chunks
      raw.mt = *(const uint4*)(pf_smem + L::OFF_HB + (H & 1) * HBS + wv * L::HB_W + r32 * 32 + 16 * j);
      // int8 scales {c0 run0, c0 run1, c1 run0, c1 run1}: chunks 2g, 2g + 1 -> bytes 4g .. 4g + 3
      raw.scw = *(const uint32_t*)(rbp + 4 * (kt & 3));
      raw.dw = *(const uint32_t*)(pf_smem + L::OFF_D + (B & 1) * DBS + wv * L::D_W + r32 * 4);
    } else {
      raw.mt = *(const uint4*)rbp;
    }
    rkt = kt;
  };
  auto dec = [&](auto sc) __attribute__((always_inline)) {
    constexpr int S4 = decltype(sc)::value;
    const int dpar = L::Q6 ? (int)(((uint32_t)(wcol0 + r32) * nbk + (uint32_t)(rkt >> 2)) & 1u) : 0;
    bf[S4] = pf_bdec32<QT, S4>(raw, h, rkt, dpar);
    asm volatile("" : "+v"(bf[S4]));  // keep the decode in this phase (else sunk past the barrier)
  };
  auto ldA = [&](const uint8_t* sl, gbf16x8(&f)[GD], int p) __attribute__((always_inline)) {
    const int sp = p / ND, g = p % ND;
#pragma unroll
    for (int i = 0; i < GD; ++i) {
      const int row = 32 * (g * GD + i) + r32;
      const uint4 av = *(const uint4*)(sl + row * 128 + (((2 * sp + h) ^ ((row >> 1) & 7)) << 4));
      __builtin_memcpy(&f[i], &av, 16);
    }
  };
  auto mfma_range = [&](const gbf16x8(&f)[GD], int p, int k0, int k1) __attribute__((always_inline)) {
    const int sp = p / ND, g = p % ND;
#pragma unroll
    for (int i = 0; i < GD; ++i)
      if (i >= k0 && i < k1)
        acc[g * GD + i] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(f[i], bf[sp], acc[g * GD + i], 0, 0, 0);
  };
  if constexpr (!(PROBE & 1)) pf_vmcnt<PW>();  // the prologue group landed (G(-2) in flight)
  read_raw(kt0);
  dec(std::integral_constant<int, 0>{});
  dec(std::integral_constant<int, 1>{});
  dec(std::integral_constant<int, 2>{});
  asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
  pf_barrier();
  ldA(pf_smem, fa, 0);

  int cur = 0;
  for (int s = 0; s < nk; ++s) {
    const uint8_t* slot = pf_smem + cur * L::A_BYTES;
    const int nxt = cur == NSA - 1 ? 0 : cur + 1;
    static_for<NPH>([&](auto pc) {
      constexpr int p = decltype(pc)::value;
      __builtin_amdgcn_sched_barrier(0);
      auto& cf = (p % 2 == 0) ? fa : fb;
      auto& nf = (p % 2 == 0) ? fb : fa;
      if constexpr (p + 1 < NPH) ldA(slot, nf, p + 1);
      if constexpr (p == 0) dec(std::integral_constant<int, 3>{});  // this step's fragment 3
      if constexpr (p == ND) {
        // G(s-2) landed (step s+1's codes / records, this wave's A pieces of it); nothing of G(s-1)
        // is issued before this point
        if constexpr (!(PROBE & 1)) pf_vmcnt<0>();
        read_raw(kt0 + s + 1);  // (past the last step: stale buffers, unused)
        dec(std::integral_constant<int, 0>{});
      }
      if constexpr (p == 2 * ND) dec(std::integral_constant<int, 1>{});
      if constexpr (ND > 1 && p == 3 * ND) dec(std::integral_constant<int, 2>{});
      if constexpr (!(PROBE & 4)) {
        if constexpr (p >= ND) group(s - 1, pc);
      }
      if constexpr (p + 1 < NPH) {
        mfma_range(cf, p, 0, GD);
      } else {
        mfma_range(cf, p, 0, GD / 2);
        __builtin_amdgcn_sched_barrier(0);
        if constexpr (ND == 1) dec(std::integral_constant<int, 2>{});
        asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
        if constexpr (!(PROBE & 8)) pf_barrier();
        ldA(pf_smem + nxt * L::A_BYTES, nf, 0);
        mfma_range(cf, p, GD / 2, GD);
      }
    });
    cur = nxt;
  }
  pf_vmcnt<0>();  // no LDS-DMA may land after this workgroup's LDS is released

  // epilogue -- C/D map of the 32x32 accumulator: col = lane & 31, row = (e & 3) + 8 (e >> 2) + 4 h
  const int n = n0 + wv * WC + r32;
#pragma unroll
  for (int i = 0; i < MT; ++i) {
#pragma unroll
    for (int e = 0; e < 16; ++e) {
      const int m = m0 + 32 * i + (e & 3) + 8 * (e >> 2) + 4 * h;
      const float v = acc[i][e];
      if constexpr (EPI == GEPI_SWIGLU_BF16) {
        const float up = __int_as_float(__builtin_amdgcn_mov_dpp(__float_as_int(v), 0xB1, 0xF, 0xF, false));
        if (m < a.M && !(r32 & 1)) a.C16[(size_t)m * a.ldc + (n >> 1)] = f32_to_bf16(glu_act(v, a.act) * up);
      } else if constexpr (EPI == GEPI_STORE16) {
        if (m < a.M) a.C16[(size_t)m * a.ldc + n] = f32_to_bf16(store16_val(a, n, v));
      } else if (m < a.M) {
        float* cp = a.C + (size_t)m * a.ldc + n;
        if (S > 1) unsafeAtomicAdd(cp, v);
        else if constexpr (EPI == GEPI_ACCUM) *cp += v;
        else *cp = v;
      }
    }
  }
}

// stacks the 256-column launches run on pf8_body (64-weight K-steps, Pf4Layout planes) instead of pf8c:
// bf16, and the Q5_K / Q4_0 / Q8_0 recipes' stacks (their Q6_K segments too)
template <int QT0, int QT1>
constexpr bool pf8_generic() {
  return QT0 == QT_BF16 || QT0 == QT_Q5_K || QT0 == QT_Q4_0 || QT0 == QT_Q8_0;
}

template <int QT0, int QT1, int BM, int EPI, int PROBE = 0>
__global__ void __launch_bounds__(512) gemm_pf8_kernel(GemmQArgs a) {
  const int nN = a.N / 256, nM = (a.M + BM - 1) / BM, total = nN * nM;
  const int L = xcd_remap(blockIdx.x, total);
  const int tn = L % nN, tm = L / nN;
  const int m0 = tm * BM, n0 = tn * 256;
  int seg = 0;
  if (a.nseg > 1 && n0 >= a.seg_n0[1]) seg = 1;
  if (a.nseg > 2 && n0 >= a.seg_n0[2]) seg = 2;
  const int S = gridDim.y;
  if constexpr (pf8_generic<QT0, QT1>()) {
    const int nk_all = a.K / 64;
    const int kt0 = (int)((long)blockIdx.y * nk_all / S), kt1 = (int)((long)(blockIdx.y + 1) * nk_all / S);
    if constexpr (QT0 != QT1) {
      if (seg == a.nseg - 1) {
        pf8_body<QT1, BM, EPI, PROBE>(a, m0, n0, seg, kt0, kt1, S);
        return;
      }
    }
    pf8_body<QT0, BM, EPI, PROBE>(a, m0, n0, seg, kt0, kt1, S);
  } else {
    // K-quant stacks: pf8c, slices on 256-block boundaries
    const int nb = a.K / 256;
    const int kt0 = 4 * (int)((long)blockIdx.y * nb / S), kt1 = 4 * (int)((long)(blockIdx.y + 1) * nb / S);
    // PROBE bit 64: the 32x32x16 body (pf8d) instead of pf8c, for A/B timing (measured slower with
    // the DMA on: gate/up M = 2048 611 vs 484 us, round 5)
    if constexpr (QT0 != QT1) {
      if (seg == a.nseg - 1) {
        if constexpr (PROBE & 64) pf8d_body<QT1, BM, EPI, PROBE>(a, m0, n0, seg, kt0, kt1, S);
        else pf8c_body<QT1, BM, EPI, PROBE>(a, m0, n0, seg, kt0, kt1, S);
        return;
      }
    }
    if constexpr (PROBE & 64) pf8d_body<QT0, BM, EPI, PROBE>(a, m0, n0, seg, kt0, kt1, S);
    else pf8c_body<QT0, BM, EPI, PROBE>(a, m0, n0, seg, kt0, kt1, S);
  }
}

// Tail split (round 5).  A 256x256-tile launch of T tiles runs one workgroup per CU (LDS), so it
// takes ceil(T / CUs) rounds; when the last round is at most half full (R = T mod CUs <= CUs / 2)
// the other CUs idle through it -- Mistral's gate/up at 2048 rows is 896 tiles = 3.5 rounds of 256
// that cost 4.  Here the first T - R tiles run as usual and each of the last R runs as TWO 128-row
// workgroups (the BM = 128 body on its half), dispatched last: the final round puts half-size work
// on every CU.  K-quant stacks, S = 1 (plans with split-K fill the chip their own way).
template <int QT0, int QT1, int EPI>
__global__ void __launch_bounds__(512) gemm_pf8t_kernel(GemmQArgs a, int F) {
  const int nN = a.N / 256;
  int L, half = -1;
  if ((int)blockIdx.x < F) {
    L = xcd_remap(blockIdx.x, F);
  } else {
    const int j = xcd_remap(blockIdx.x - F, gridDim.x - F);
    L = F + (j >> 1);
    half = j & 1;
  }
  const int tn = L % nN, tm = L / nN;
  const int m0 = tm * 256 + (half > 0 ? 128 : 0), n0 = tn * 256;
  int seg = 0;
  if (a.nseg > 1 && n0 >= a.seg_n0[1]) seg = 1;
  if (a.nseg > 2 && n0 >= a.seg_n0[2]) seg = 2;
  const int kt1 = 4 * (a.K / 256);
  if constexpr (pf8_generic<QT0, QT1>()) {
    if constexpr (QT0 != QT1) {
      if (seg == a.nseg - 1) {
        if (half < 0) pf8_body<QT1, 256, EPI>(a, m0, n0, seg, 0, kt1, 1);
        else pf8_body<QT1, 128, EPI>(a, m0, n0, seg, 0, kt1, 1);
        return;
      }
    }
    if (half < 0) pf8_body<QT0, 256, EPI>(a, m0, n0, seg, 0, kt1, 1);
    else pf8_body<QT0, 128, EPI>(a, m0, n0, seg, 0, kt1, 1);
  } else {
    if constexpr (QT0 != QT1) {
      if (seg == a.nseg - 1) {
        if (half < 0) pf8c_body<QT1, 256, EPI>(a, m0, n0, seg, 0, kt1, 1);
        else pf8c_body<QT1, 128, EPI>(a, m0, n0, seg, 0, kt1, 1);
        return;
      }
    }
    if (half < 0) pf8c_body<QT0, 256, EPI>(a, m0, n0, seg, 0, kt1, 1);
    else pf8c_body<QT0, 128, EPI>(a, m0, n0, seg, 0, kt1, 1);
  }
}

// full tiles before the tail of a 256 x BN launch, or -1 (no tail split for this shape / plan)
inline int pf_tail_full(const GemmQArgs& a, int BN, int S) {
  const char* e = std::getenv("AIOS_GEMM_PF_TAIL");  // (read per call: tests compare both)
  if ((e && std::atoi(e) == 0) || S != 1 || a.epi == GEPI_QKV || a.epi == GEPI_STORE16) return -1;
  const int T = (a.N / BN) * ((a.M + 255) / 256), C = device_cu_count(), R = T % C;
  return (T > C && R > 0 && 2 * R <= C) ? T - R : -1;
}

// Stream-K (round 6): a launch whose output tiles do not fill the chip -- the N = 4096-6144
// projections of a 512-token chunk have 32-192 tiles for 256 CUs -- runs one workgroup per CU over an
// equal share of the flattened (tile, K-step) iteration space instead of split-K's equal slices of
// every tile: workgroup w takes iterations [w * ipw, (w + 1) * ipw), i.e. the tail of one tile and the
// head of the next, and adds each partial tile into C with the split-K atomics (STORE targets zeroed
// first).  KG: K-steps per unit (4 for the K-quant pf8c body, which slices on 256-blocks).  A workgroup
// that runs a second segment barriers first: the previous body's last LDS reads against its prologue DMA.
template <int QT0, int QT1, int BM, int EPI, int KG, typename Body>
__device__ __forceinline__ void pf_stream_k(const GemmQArgs& a, int BN, int ipw, Body body) {
  const int nN = a.N / BN, nM = (a.M + BM - 1) / BM;
  const int nk = a.K / (64 * KG);
  const long total = (long)nN * nM * nk;
  long it = (long)blockIdx.x * ipw;
  const long end = it + ipw < total ? it + ipw : total;
  bool first = true;
  while (it < end) {
    const int L = (int)(it / nk), k0 = (int)(it - (long)L * nk);
    const int k1 = (int)(k0 + (end - it) < nk ? k0 + (end - it) : nk);
    const int tn = L % nN, tm = L / nN;
    const int m0 = tm * BM, n0 = tn * BN;
    int seg = 0;
    if (a.nseg > 1 && n0 >= a.seg_n0[1]) seg = 1;
    if (a.nseg > 2 && n0 >= a.seg_n0[2]) seg = 2;
    if (!first) __syncthreads();
    // S: 1 when this workgroup owns the whole tile (plain epilogue), else atomic partials
    body(m0, n0, seg, k0 * KG, k1 * KG, (k0 == 0 && k1 == nk) ? 1 : 2);
    it += k1 - k0;
    first = false;
  }
}

template <int QT0, int QT1, int BM, int WC, int EPI>
__global__ void __launch_bounds__(256) gemm_pf4sk_kernel(GemmQArgs a, int ipw) {
  pf_stream_k<QT0, QT1, BM, EPI, 1>(a, 4 * WC, ipw, [&](int m0, int n0, int seg, int kt0, int kt1, int S) {
    if constexpr (QT0 != QT1) {
      if (seg == a.nseg - 1) {
        pf4_body<QT1, BM, WC, EPI>(a, m0, n0, seg, kt0, kt1, S);
        return;
      }
    }
    pf4_body<QT0, BM, WC, EPI>(a, m0, n0, seg, kt0, kt1, S);
  });
}

template <int QT0, int QT1, int BM, int EPI>
__global__ void __launch_bounds__(512) gemm_pf8sk_kernel(GemmQArgs a, int ipw) {
  constexpr int KG = pf8_generic<QT0, QT1>() ? 1 : 4;
  pf_stream_k<QT0, QT1, BM, EPI, KG>(a, 256, ipw, [&](int m0, int n0, int seg, int kt0, int kt1, int S) {
    if constexpr (pf8_generic<QT0, QT1>()) {
      if constexpr (QT0 != QT1) {
        if (seg == a.nseg - 1) {
          pf8_body<QT1, BM, EPI>(a, m0, n0, seg, kt0, kt1, S);
          return;
        }
      }
      pf8_body<QT0, BM, EPI>(a, m0, n0, seg, kt0, kt1, S);
    } else {
      if constexpr (QT0 != QT1) {
        if (seg == a.nseg - 1) {
          pf8c_body<QT1, BM, EPI>(a, m0, n0, seg, kt0, kt1, S);
          return;
        }
      }
      pf8c_body<QT0, BM, EPI>(a, m0, n0, seg, kt0, kt1, S);
    }
  });
}

// iterations per workgroup of a stream-K launch over the device's CUs (workgroups = its grid)
inline int pf_sk_ipw(const GemmQArgs& a, int BM, int BN, int KG, int& grid) {
  const long total = (long)(a.N / BN) * ((a.M + BM - 1) / BM) * (a.K / (64 * KG));
  const int cus = device_cu_count();
  // (even: with an even K-step count per tile every segment is >= 2 units, as the split-K slices)
  const int ipw = (int)(((total + cus - 1) / cus + 1) & ~1L);
  grid = (int)((total + ipw - 1) / ipw);
  return ipw;
}

template <int QT0, int QT1, int BM>
constexpr int pf8_lds_bytes() {
  if constexpr (pf8_generic<QT0, QT1>()) {
    using L0 = Pf4Layout<QT0, BM, 32, 8>;
    using L1 = Pf4Layout<QT1, BM, 32, 8>;
    return L0::NS * L0::SLOT > L1::NS * L1::SLOT ? L0::NS * L0::SLOT : L1::NS * L1::SLOT;
  } else {
    return PfcLayout<QT0, BM>::TOTAL > PfcLayout<QT1, BM>::TOTAL ? PfcLayout<QT0, BM>::TOTAL
                                                                 : PfcLayout<QT1, BM>::TOTAL;
  }
}

template <int QT0, int QT1, int BM>
void pf8_launch(const GemmQArgs& a, int S, hipStream_t st) {
  constexpr int lds = pf8_lds_bytes<QT0, QT1, BM>();
  static_assert(lds <= 160 * 1024, "LDS");
  if (S < 0) {  // stream-K (STORE / ACCUM only: partial tiles are atomic adds)
    int grid = 0;
    const int ipw = pf_sk_ipw(a, BM, 256, pf8_generic<QT0, QT1>() ? 1 : 4, grid);
    if (a.epi == GEPI_STORE)
      hipLaunchKernelGGL((gemm_pf8sk_kernel<QT0, QT1, BM, GEPI_STORE>), dim3(grid), dim3(512), lds, st, a, ipw);
    else
      hipLaunchKernelGGL((gemm_pf8sk_kernel<QT0, QT1, BM, GEPI_ACCUM>), dim3(grid), dim3(512), lds, st, a, ipw);
    return;
  }
  if constexpr (BM == 256 && QT0 != QT_BF16) {  // (K-quant stacks: the tail split)
    const int F = pf_tail_full(a, 256, S);
    if (F >= 0) {
      constexpr int l128 = pf8_lds_bytes<QT0, QT1, 128>();
      constexpr int ldst = lds > l128 ? lds : l128;
      const int T = (a.N / 256) * ((a.M + 255) / 256);
      const dim3 grid(F + 2 * (T - F)), block(512);
      switch (a.epi) {
        case GEPI_STORE: hipLaunchKernelGGL((gemm_pf8t_kernel<QT0, QT1, GEPI_STORE>), grid, block, ldst, st, a, F); break;
        case GEPI_ACCUM: hipLaunchKernelGGL((gemm_pf8t_kernel<QT0, QT1, GEPI_ACCUM>), grid, block, ldst, st, a, F); break;
        default: hipLaunchKernelGGL((gemm_pf8t_kernel<QT0, QT1, GEPI_SWIGLU_BF16>), grid, block, ldst, st, a, F); break;
      }
      return;
    }
  }
  const dim3 grid((a.N / 256) * ((a.M + BM - 1) / BM), S), block(512);
  switch (a.epi) {
    case GEPI_STORE: hipLaunchKernelGGL((gemm_pf8_kernel<QT0, QT1, BM, GEPI_STORE>), grid, block, lds, st, a); break;
    case GEPI_ACCUM: hipLaunchKernelGGL((gemm_pf8_kernel<QT0, QT1, BM, GEPI_ACCUM>), grid, block, lds, st, a); break;
    case GEPI_QKV: hipLaunchKernelGGL((gemm_pf8_kernel<QT0, QT1, BM, GEPI_QKV>), grid, block, lds, st, a); break;
    case GEPI_STORE16:
      if constexpr (QT0 == QT_BF16) hipLaunchKernelGGL((gemm_pf8_kernel<QT0, QT1, BM, GEPI_STORE16>), grid, block, lds, st, a);
      break;
    default: hipLaunchKernelGGL((gemm_pf8_kernel<QT0, QT1, BM, GEPI_SWIGLU_BF16>), grid, block, lds, st, a); break;
  }
}

template <int QT0, int QT1, int BM, int WC, int EPI, int PROBE = 0>
__global__ void __launch_bounds__(256) gemm_pf4_kernel(GemmQArgs a) {
  constexpr int BN = 4 * WC;
  const int nN = a.N / BN, nM = (a.M + BM - 1) / BM, total = nN * nM;
  const int L = xcd_remap(blockIdx.x, total);
  const int tn = L % nN, tm = L / nN;
  const int m0 = tm * BM, n0 = tn * BN;
  int seg = 0;
  if (a.nseg > 1 && n0 >= a.seg_n0[1]) seg = 1;
  if (a.nseg > 2 && n0 >= a.seg_n0[2]) seg = 2;
  const int S = gridDim.y, nk_all = a.K / 64;
  const int kt0 = (int)((long)blockIdx.y * nk_all / S), kt1 = (int)((long)(blockIdx.y + 1) * nk_all / S);
  if constexpr (QT0 != QT1) {
    if (seg == a.nseg - 1) {
      pf4_body<QT1, BM, WC, EPI, PROBE>(a, m0, n0, seg, kt0, kt1, S);
      return;
    }
  }
  pf4_body<QT0, BM, WC, EPI, PROBE>(a, m0, n0, seg, kt0, kt1, S);
}

// pf4's tail split (256 x 4 WC tiles): as gemm_pf8t_kernel, the last R tiles as two 128-row halves
template <int QT0, int QT1, int WC, int EPI>
__global__ void __launch_bounds__(256) gemm_pf4t_kernel(GemmQArgs a, int F) {
  constexpr int BN = 4 * WC;
  const int nN = a.N / BN;
  int L, half = -1;
  if ((int)blockIdx.x < F) {
    L = xcd_remap(blockIdx.x, F);
  } else {
    const int j = xcd_remap(blockIdx.x - F, gridDim.x - F);
    L = F + (j >> 1);
    half = j & 1;
  }
  const int tn = L % nN, tm = L / nN;
  const int m0 = tm * 256 + (half > 0 ? 128 : 0), n0 = tn * BN;
  int seg = 0;
  if (a.nseg > 1 && n0 >= a.seg_n0[1]) seg = 1;
  if (a.nseg > 2 && n0 >= a.seg_n0[2]) seg = 2;
  const int kt1 = a.K / 64;
  if constexpr (QT0 != QT1) {
    if (seg == a.nseg - 1) {
      if (half < 0) pf4_body<QT1, 256, WC, EPI>(a, m0, n0, seg, 0, kt1, 1);
      else pf4_body<QT1, 128, WC, EPI>(a, m0, n0, seg, 0, kt1, 1);
      return;
    }
  }
  if (half < 0) pf4_body<QT0, 256, WC, EPI>(a, m0, n0, seg, 0, kt1, 1);
  else pf4_body<QT0, 128, WC, EPI>(a, m0, n0, seg, 0, kt1, 1);
}

template <int QT0, int QT1, int BM, int WC>
constexpr int pf4_lds_bytes() {
  using L0 = Pf4Layout<QT0, BM, WC>;
  using L1 = Pf4Layout<QT1, BM, WC>;
  return L0::NS * L0::SLOT > L1::NS * L1::SLOT ? L0::NS * L0::SLOT : L1::NS * L1::SLOT;
}

template <int QT0, int QT1, int BM, int WC>
void pf4_launch(const GemmQArgs& a, int S, hipStream_t st) {
  constexpr int lds = pf4_lds_bytes<QT0, QT1, BM, WC>();
  static_assert(lds <= 160 * 1024, "LDS");
  if (S < 0) {  // stream-K (STORE / ACCUM only)
    int grid = 0;
    const int ipw = pf_sk_ipw(a, BM, 4 * WC, 1, grid);
    if (a.epi == GEPI_STORE)
      hipLaunchKernelGGL((gemm_pf4sk_kernel<QT0, QT1, BM, WC, GEPI_STORE>), dim3(grid), dim3(256), lds, st, a, ipw);
    else
      hipLaunchKernelGGL((gemm_pf4sk_kernel<QT0, QT1, BM, WC, GEPI_ACCUM>), dim3(grid), dim3(256), lds, st, a, ipw);
    return;
  }
  if constexpr (BM == 256) {
    const int F = pf_tail_full(a, 4 * WC, S);
    if (F >= 0) {
      constexpr int l128 = pf4_lds_bytes<QT0, QT1, 128, WC>();
      constexpr int ldst = lds > l128 ? lds : l128;
      const int T = (a.N / (4 * WC)) * ((a.M + 255) / 256);
      const dim3 grid(F + 2 * (T - F)), block(256);
      switch (a.epi) {
        case GEPI_STORE: hipLaunchKernelGGL((gemm_pf4t_kernel<QT0, QT1, WC, GEPI_STORE>), grid, block, ldst, st, a, F); break;
        case GEPI_ACCUM: hipLaunchKernelGGL((gemm_pf4t_kernel<QT0, QT1, WC, GEPI_ACCUM>), grid, block, ldst, st, a, F); break;
        default: hipLaunchKernelGGL((gemm_pf4t_kernel<QT0, QT1, WC, GEPI_SWIGLU_BF16>), grid, block, ldst, st, a, F); break;
      }
      return;
    }
  }
  const dim3 grid((a.N / (4 * WC)) * ((a.M + BM - 1) / BM), S), block(256);
  switch (a.epi) {
    case GEPI_STORE: hipLaunchKernelGGL((gemm_pf4_kernel<QT0, QT1, BM, WC, GEPI_STORE>), grid, block, lds, st, a); break;
    case GEPI_ACCUM: hipLaunchKernelGGL((gemm_pf4_kernel<QT0, QT1, BM, WC, GEPI_ACCUM>), grid, block, lds, st, a); break;
    case GEPI_QKV: hipLaunchKernelGGL((gemm_pf4_kernel<QT0, QT1, BM, WC, GEPI_QKV>), grid, block, lds, st, a); break;
    case GEPI_STORE16:
      if constexpr (QT0 == QT_BF16) hipLaunchKernelGGL((gemm_pf4_kernel<QT0, QT1, BM, WC, GEPI_STORE16>), grid, block, lds, st, a);
      break;
    default: hipLaunchKernelGGL((gemm_pf4_kernel<QT0, QT1, BM, WC, GEPI_SWIGLU_BF16>), grid, block, lds, st, a); break;
  }
}

// One launch for every tile of a (possibly mixed-format) segment stack: tiles of the last segment
// run the QT1 body (the Q4_K_M QKV stack: Q|K Q4_K, V Q6_K).  gridDim.y = K slices (atomic adds).
#ifndef AIOS_PF_MF
#define AIOS_PF_MF 32  // MFMA shape of the production body (16: the 16x16x32 body)
#endif
template <int QT0, int QT1, int BM, int NW, int NS, int EPI, int PROBE = 0, int MF = AIOS_PF_MF>
__global__ void __launch_bounds__(NW * 64) gemm_pf_kernel(GemmQArgs a) {
  constexpr int BN = NW * 32;
  const int nN = a.N / BN, nM = (a.M + BM - 1) / BM, total = nN * nM;
  const int L = xcd_remap(blockIdx.x, total);
  const int tn = L % nN, tm = L / nN;
  const int m0 = tm * BM, n0 = tn * BN;
  int seg = 0;
  if (a.nseg > 1 && n0 >= a.seg_n0[1]) seg = 1;
  if (a.nseg > 2 && n0 >= a.seg_n0[2]) seg = 2;
  const int S = gridDim.y, nk_all = a.K / 64;
  const int kt0 = (int)((long)blockIdx.y * nk_all / S), kt1 = (int)((long)(blockIdx.y + 1) * nk_all / S);
  if constexpr (QT0 != QT1) {
    if (seg == a.nseg - 1) {
      if constexpr (MF == 32) pf_body32<QT1, BM, NW, NS, EPI, PROBE>(a, m0, n0, seg, kt0, kt1, S);
      else pf_body<QT1, BM, NW, NS, EPI, PROBE>(a, m0, n0, seg, kt0, kt1, S);
      return;
    }
  }
  if constexpr (MF == 32) pf_body32<QT0, BM, NW, NS, EPI, PROBE>(a, m0, n0, seg, kt0, kt1, S);
  else pf_body<QT0, BM, NW, NS, EPI, PROBE>(a, m0, n0, seg, kt0, kt1, S);
}

// slot bytes of a launch (the larger format's) and its slot count: 3 where they fit in 160 KB
template <int QT0, int QT1, int BM, int NW>
constexpr int pf_slot_bytes() {
  return PfLayout<QT0, BM, NW * 32>::SLOT > PfLayout<QT1, BM, NW * 32>::SLOT ? PfLayout<QT0, BM, NW * 32>::SLOT
                                                                             : PfLayout<QT1, BM, NW * 32>::SLOT;
}
template <int QT0, int QT1, int BM, int NW>
constexpr int pf_slots() {
  return 3 * pf_slot_bytes<QT0, QT1, BM, NW>() <= 160 * 1024 ? 3 : 2;
}

// host: launch one instantiation (grid = tiles x S)
template <int QT0, int QT1, int BM, int NW>
void pf_launch(const GemmQArgs& a, int S, hipStream_t st) {
  constexpr int BN = NW * 32;
  constexpr int NS = pf_slots<QT0, QT1, BM, NW>();
  constexpr int lds = NS * pf_slot_bytes<QT0, QT1, BM, NW>();
  static_assert(lds <= 160 * 1024, "LDS");
  const dim3 grid((a.N / BN) * ((a.M + BM - 1) / BM), S), block(NW * 64);
  switch (a.epi) {
    case GEPI_STORE: hipLaunchKernelGGL((gemm_pf_kernel<QT0, QT1, BM, NW, NS, GEPI_STORE>), grid, block, lds, st, a); break;
    case GEPI_ACCUM: hipLaunchKernelGGL((gemm_pf_kernel<QT0, QT1, BM, NW, NS, GEPI_ACCUM>), grid, block, lds, st, a); break;
    default: hipLaunchKernelGGL((gemm_pf_kernel<QT0, QT1, BM, NW, NS, GEPI_SWIGLU_BF16>), grid, block, lds, st, a); break;
  }
}

// the tile set of one format pair (one translation unit each, compiled in parallel): BM x BN tiles,
// BN = 4 waves x WC columns
template <int QT0, int QT1>
bool pf_launch_fmt(const GemmQArgs& a, int BM, int BN, int S, hipStream_t st) {
  // 256-column tiles: the 8-wave body (pf8 / pf8c); 128-column tiles: pf4 with 32 columns per wave
#define PF_GO8(bm)                      \
  if (BM == bm && BN == 256) {          \
    pf8_launch<QT0, QT1, bm>(a, S, st); \
    return true;                        \
  }
#define PF_GO4(bm)                          \
  if (BM == bm && BN == 128) {              \
    pf4_launch<QT0, QT1, bm, 32>(a, S, st); \
    return true;                            \
  }
  PF_GO8(256) PF_GO8(128) PF_GO8(64) PF_GO4(256) PF_GO4(128) PF_GO4(64)
#undef PF_GO8
#undef PF_GO4
  return false;
}

}  // namespace aios
