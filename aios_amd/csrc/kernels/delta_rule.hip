// The gated delta rule (mixers.h LIN_DELTA): per head S_t = d_t S_{t-1} + k_t u_t^T, u_t = b_t (v_t - d_t S_{t-1}^T k_t),
// o_t = S_t^T q_t, with unit k and q.
//
// Portions, in pairs of 16-token blocks (a pair is one ScanChunk), after the convolution of linear_scan.hip and before its norm:
//   score   With D_t the decay since the pair's start and S the state there, the pair's u solve
//             u_t + b_t sum_{s<t} (D_t / D_s) (k_t . k_s) u_s = b_t (v_t - D_t S^T k_t):
//           block by block a unit lower-triangular system, whose inverse times diag(b) is a 16 x 16 matrix T that does not
//           depend on S.  Left for the walk: T of both blocks, the block-to-block part of the system, and the scores
//           (D_t / D_s) q_t . k_s, s <= t.  k and q are kept as the convolution left them; their lengths are numbers per token
//           that go with the decays and into these matrices.
//   walk    a wave owns a head and 16 columns of v, its part of S in accumulators from pair to pair:
//             u = T (v - D K S - ..),  o = D Q S + scores u,  S = (decay of the pair) S + K^T (decay to its end) u.
//           A 16 x 16 accumulator tile is, lane for lane, the second operand of the 16-deep product, so neither S nor u
//           leaves registers.  Where heads and columns leave compute units idle, a portion is walked in segments side by side: a
//           segment's transition S -> M S + E is the walk of the unit matrix without values and the walk from zero, so a first
//           walk finds M and E of all segments but the last, the second one starts each from what those before it make together.
// Single tokens: delta_step, one workgroup per head and row, the norm included.
//
// fp32: state, decays, strengths, lengths, the system and its inverse, scores, norms, gates.  The products take bf16 operands:
// q, k, v as the convolution left them; the state, u and every matrix of the pair as two bf16 terms (hi + lo).  The 32-bit form
// (F32) runs the same steps on fp32 matrix instructions.
#include <algorithm>
#include <stdexcept>

#include "lin_common.h"

namespace aios {

// what score leaves for a pair and head: matrices, row-major [t][s] (bf16: hi, then lo) ...
enum DeltaMat { DM_A0 = 0, DM_A1 = 1, DM_A10 = 2, DM_T0 = 3, DM_T1 = 4, DM_L10 = 5, DM_N = 6 };
// ... and numbers: per block [16] the decay since the pair's start times q's factor, the decay to its end times k's, the decay
// since its start times k's; then the decay of the pair
constexpr int DD_BLOCK = 48, DD_TOT = 96, DD_N = 128;

// eight numbers of a lane: two tiles' depths 4 q + r (bf16: 16 bytes)
template <bool F32>
struct Oct {
  gf32x4 a, b;
};
template <>
struct Oct<false> {
  gu32x4 u;
};
template <bool F32>
__device__ __forceinline__ Oct<F32> oct(const void* base, size_t at) {
  if constexpr (F32) return Oct<F32>{*(const gf32x4*)((const float*)base + at), *(const gf32x4*)((const float*)base + at + 4)};
  else return Oct<F32>{*(const gu32x4*)((const bf16_t*)base + at)};
}
// c + (both tiles of x) times (both tiles of y)
__device__ __forceinline__ gf32x4 mul8(const Oct<false>& x, const Oct<false>& y, gf32x4 c) {
  return __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(gbf16x8, x.u), __builtin_bit_cast(gbf16x8, y.u), c, 0, 0, 0);
}
__device__ __forceinline__ gf32x4 mul8(const Oct<true>& x, const Oct<true>& y, gf32x4 c) { return mfma4(x.b, y.b, mfma4(x.a, y.a, c)); }
__device__ __forceinline__ Oct<false> join(lu2 a, lu2 b) { return Oct<false>{gu32x4{a.x, a.y, b.x, b.y}}; }

// a tile of accumulators as an operand: as it is (F32), or hi and lo
template <bool F32>
struct Tile {
  gf32x4 f;
};
template <>
struct Tile<false> {
  lu2 h, l;
};
template <bool F32>
__device__ __forceinline__ Tile<F32> tile(gf32x4 f) {
  Tile<F32> x;
  if constexpr (F32) x.f = f;
  else split4(f, x.h, x.l);
  return x;
}

// a pair's matrix, [t][s]: bf16 as hi and lo of four s beside each other
template <bool F32>
struct Mat {
  gf32x4 f;
};
template <>
struct Mat<false> {
  gu32x4 u;  // hi, lo
};
constexpr int mat_size(bool f32) { return f32 ? 256 : 512; }
template <bool F32>
__device__ __forceinline__ size_t mat_at(int t, int s) { return F32 ? t * 16 + s : t * 32 + (s >> 2) * 8 + (s & 3); }
template <bool F32>
__device__ __forceinline__ Mat<F32> mat(const void* so, size_t at) {
  if constexpr (F32) return Mat<F32>{*(const gf32x4*)((const float*)so + at)};
  else return Mat<F32>{*(const gu32x4*)((const bf16_t*)so + at)};
}
template <bool F32>
__device__ __forceinline__ void put_mat(void* so, size_t at, gf32x4 v) {
  if constexpr (F32) {
    *(gf32x4*)((float*)so + at) = v;
  } else {
    lu2 hi, lo;
    split4(v, hi, lo);
    *(gu32x4*)((bf16_t*)so + at) = gu32x4{hi.x, hi.y, lo.x, lo.y};
  }
}
// c + m x
__device__ __forceinline__ gf32x4 mul(const Mat<true>& m, const Tile<true>& x, gf32x4 c) { return mfma4(m.f, x.f, c); }
__device__ __forceinline__ gf32x4 mul(const Mat<false>& m, const Tile<false>& x, gf32x4 c) {
  const Oct<false> o{m.u};
  return mul8(o, join(x.h, x.h), mul8(o, join(x.l, x.l), c));
}
// c + x's two tiles times s and t
__device__ __forceinline__ gf32x4 mul(const Oct<true>& x, const Tile<true>& s, const Tile<true>& t, gf32x4 c) {
  return mfma4(x.b, t.f, mfma4(x.a, s.f, c));
}
__device__ __forceinline__ gf32x4 mul(const Oct<false>& x, const Tile<false>& s, const Tile<false>& t, gf32x4 c) {
  return mul8(x, join(s.h, t.h), mul8(x, join(s.l, t.l), c));
}

static_assert(SCAN_CHUNK == 2 * LIN_T, "a pair of blocks is a chunk");

// a wave per (pair, head)
template <bool F32>
__global__ void __launch_bounds__(256) delta_score_kernel(LinScanArgs a, int nscore, int nkeep) {
  if ((int)blockIdx.x >= nscore) return lin_keep(a, blockIdx.x - nscore, nkeep);
  __shared__ float sl[4][16][20];
  const int lane = threadIdx.x & 63, idx = blockIdx.x * 4 + (threadIdx.x >> 6);
  const int pair = idx / a.H, h = idx - pair * a.H;
  if (pair >= a.n_chunks) return;
  const ScanChunk ch = a.chunks[pair];
  const int r16 = lane & 15, q = lane >> 4;
  // token r16 of both blocks: log decay since the pair's start, strength
  const float e = expf(a.a_log[h]);
  float cum[2], beta[2];
#pragma unroll
  for (int b = 0; b < 2; ++b) {
    const int t = 16 * b + r16;
    const float* in = a.in + (size_t)(ch.row0 + t) * a.ld;
    cum[b] = beta[b] = 0.f;
    if (t < ch.n) {
      cum[b] = -e * ls_softplus(in[a.dt_off + h] + a.dt_b[h]);
      beta[b] = 1.f / (1.f + expf(-in[a.b_off + h]));
    }
#pragma unroll
    for (int d = 1; d < 16; d <<= 1) {
      const float o = __shfl_up(cum[b], d, 16);
      if (r16 >= d) cum[b] += o;
    }
  }
  cum[1] += __shfl(cum[0], 15, 16);
  const float tot = __shfl(cum[1], 15, 16);
  // products of keys and queries: [s][t], a lane holds s = 4 q + r, t = r16 (s of the first, t of the second: block 1 beside 0)
  constexpr gf32x4 zero = {0.f, 0.f, 0.f, 0.f};
  gf32x4 kk[2] = {zero, zero}, qq[2] = {zero, zero}, kq[2] = {zero, zero}, kk10 = zero, kq10 = zero;
  const size_t g = h / (a.H / a.G), base = ((size_t)2 * pair * a.G + g) * a.np * 16 + r16 * 32 + 8 * q, next = (size_t)a.G * a.np * 16;
  for (int i = 0; i < a.np / 32; ++i) {
    Oct<F32> k[2], x[2];
#pragma unroll
    for (int b = 0; b < 2; ++b) {
      k[b] = oct<F32>(a.kr, base + b * next + (size_t)i * 512);
      x[b] = oct<F32>(a.qo, base + b * next + (size_t)i * 512);
    }
#pragma unroll
    for (int b = 0; b < 2; ++b) {
      kk[b] = mul8(k[b], k[b], kk[b]);
      qq[b] = mul8(x[b], x[b], qq[b]);
      kq[b] = mul8(k[b], x[b], kq[b]);
    }
    kk10 = mul8(k[0], k[1], kk10);
    kq10 = mul8(k[0], x[1], kq10);
  }
  // factors that make the token's key and query unit vectors (the query's with its scale): from the diagonals
  float ik[2], iq[2];
  float* dec = a.dec + ((size_t)pair * a.H + h) * DD_N;
#pragma unroll
  for (int b = 0; b < 2; ++b) {
    float nk = 0.f, nq = 0.f;
#pragma unroll
    for (int r = 0; r < 4; ++r)
      if (4 * q + r == r16) {
        nk = kk[b][r];
        nq = qq[b][r];
      }
    const int diag = (r16 >> 2) * 16 + r16;
    ik[b] = 1.f / sqrtf(__shfl(nk, diag, 64) + LIN_UNIT_EPS);
    iq[b] = a.q_scale / sqrtf(__shfl(nq, diag, 64) + LIN_UNIT_EPS);
    if (q == 0) {
      const float d = expf(cum[b]);
      dec[b * DD_BLOCK + r16] = iq[b] * d;
      dec[b * DD_BLOCK + 16 + r16] = ik[b] * expf(tot - cum[b]);
      dec[b * DD_BLOCK + 32 + r16] = ik[b] * d;
    }
  }
  if (lane == 0) dec[DD_TOT] = expf(tot);
  constexpr int MAT = mat_size(F32);
  const size_t so = ((size_t)pair * a.H + h) * DM_N * MAT, at = so + mat_at<F32>(r16, 4 * q);
  // block to block
  gf32x4 l, s;
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    const float d = __shfl(ik[0], 4 * q + r, 16) * expf(cum[1] - __shfl(cum[0], 4 * q + r, 16));
    l[r] = -kk10[r] * d * ik[1];  // (the walk adds it; T has the strength)
    s[r] = kq10[r] * d * iq[1];
  }
  put_mat<F32>(a.so, at + DM_L10 * MAT, l);
  put_mat<F32>(a.so, at + DM_A10 * MAT, s);
  float(*low)[20] = sl[threadIdx.x >> 6];
#pragma unroll
  for (int b = 0; b < 2; ++b) {
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const int t = 4 * q + r;
      const float d = t <= r16 ? __shfl(ik[b], t, 16) * expf(cum[b] - __shfl(cum[b], t, 16)) : 0.f;
      s[r] = kq[b][r] * d * iq[b];
      l[r] = t < r16 ? kk[b][r] * d * ik[b] * beta[b] : 0.f;
    }
    put_mat<F32>(a.so, at + (DM_A0 + b) * MAT, s);
    // column r16 of (I + l)^-1, row after row.  (A wave's slice of LDS is its own and LDS executes a wave's accesses in order;
    // the fences keep the compiler to it.)
    __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
    *(gf32x4*)(low[r16] + 4 * q) = l;
    __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
    float x[16];
#pragma unroll
    for (int i = 0; i < 16; ++i) {
      x[i] = i == r16 ? 1.f : 0.f;
#pragma unroll
      for (int j = 0; j < i; ++j) x[i] = fmaf(-low[i][j], x[j], x[i]);
    }
    const size_t tm = so + (DM_T0 + b) * MAT;
#pragma unroll
    for (int i = 0; i < 16; ++i)
      if (i >> 2 == q) {
        const float v = x[i] * beta[b];
        put1<F32>(a.so, tm + mat_at<F32>(i, r16), v);
        if constexpr (!F32) put1<F32>(a.so, tm + mat_at<F32>(i, r16) + 4, v - bf16_to_f32(f32_to_bf16(v)));
      }
  }
}

// ---- the walk ---------------------------------------------------------------------------------------
// the pairs of a portion that a segment walks: [i0, i1), and how many segments there are
constexpr int DELTA_SEG_MIN = 4;
struct DeltaSeg {
  int i0, i1, n;
};
__device__ __forceinline__ DeltaSeg delta_seg(int pairs, int nseg, int seg) {
  const int per = max(DELTA_SEG_MIN, (pairs + nseg - 1) / nseg);
  return DeltaSeg{seg * per, min(pairs, (seg + 1) * per), (pairs + per - 1) / per};
}

// Registers hold one pair's operands; each is requested anew as soon as the walk is through with it, half a step before it is
// needed again.
// ENDS: the first walk of a portion in segments, without outputs.  Segment s leaves what it ends with at seg[s + 1]: the first
// one from the state it starts from (which it copies to seg[0]), the others from zero; waves of 16 more columns each take the
// columns of the unit matrix, without values, to the segment's transition, at seg_dec[s + 1].
template <bool F32, int NT, bool ENDS>
__global__ void __launch_bounds__(64) __attribute__((amdgpu_waves_per_eu(!F32 && NT <= 8 ? 2 : 1))) delta_walk_kernel(LinScanArgs a) {
  constexpr int NP = 16 * NT, MAT = mat_size(F32);
  const int lane = threadIdx.x, nvt = a.vp >> 4, per_head = nvt + (ENDS ? NT : 0), waves = a.H * per_head;
  // (workgroups are dealt round-robin: a head's go to one XCD)
  const int per_xcd = gridDim.x >> 3, w = (blockIdx.x & 7) * per_xcd + (blockIdx.x >> 3);
  if (w >= waves) return;
  const int h = w / per_head, wt = w - h * per_head, g = h / (a.H / a.G), seg = blockIdx.z;
  const bool unit = wt >= nvt;
  const int r16 = lane & 15, q = lane >> 4;
  const ScanSeq sq = a.seqs[blockIdx.y];
  const DeltaSeg sg = delta_seg((sq.n + 2 * LIN_T - 1) / (2 * LIN_T), a.nseg, seg);
  if (seg + (ENDS ? 1 : 0) >= sg.n || (ENDS && unit && seg == 0)) return;
  const int p0 = sq.b0 / 2, col = 16 * (unit ? wt - nvt : wt) + r16;
  const size_t hs = (size_t)a.np * a.vp, half = (size_t)a.slots * a.H * hs;
  const size_t lane_at = (size_t)(4 * q) * a.vp + col;  // of this lane in a head's state
  float* st = a.state + ((size_t)sq.slot * a.H + h) * hs + lane_at;
  // segment j of this portion and head
  auto seg_at = [&](int j) { return a.seg + (((size_t)blockIdx.y * a.nseg + j) * a.H + h) * hs + lane_at; };
  auto mat_of = [&](int j) { return a.seg_dec + (((size_t)blockIdx.y * a.nseg + j) * a.H + h) * NP * NP; };
  constexpr bool HOLD = !F32 || NT <= 8;  // (what registers have room for; else operands are read where they are used)
  Oct<F32> kr[2][HOLD ? NT / 2 : 1], x[2][HOLD ? NT / 2 : 1], k[HOLD ? NT : 1], vo;
  Mat<F32> m[DM_N];
  gf32x4 d[2][3];
  float tot;
  auto pair_of = [&](int i) { return (size_t)(p0 + min(i, sg.i1 - 1)); };  // (past the end: re-reads)
  auto row_at = [&](size_t p, int b, int t) { return ((2 * p + b) * a.G + g) * NP * 16 + r16 * 32 + 8 * q + 256 * t; };
  auto col_at = [&](size_t p, int t) { return ((p * a.G + g) * NP + 16 * t + r16) * 32 + 8 * q; };
  auto load_rows = [&](int i) __attribute__((always_inline)) {
    if constexpr (!HOLD) return;
    const size_t p = pair_of(i);
#pragma unroll
    for (int t = 0; t < NT; t += 2)
#pragma unroll
      for (int b = 0; b < 2; ++b) {
        kr[b][t / 2] = oct<F32>(a.kr, row_at(p, b, t));
        if constexpr (!ENDS) x[b][t / 2] = oct<F32>(a.qo, row_at(p, b, t));
      }
  };
  auto load_rest = [&](int i) __attribute__((always_inline)) {
    const size_t p = pair_of(i);
    if (!ENDS || !unit) vo = oct<F32>(a.vo, ((p * a.H + h) * a.vp + col) * 32 + 8 * q);
    const float* dec = a.dec + (p * a.H + h) * DD_N;
#pragma unroll
    for (int b = 0; b < 2; ++b)
#pragma unroll
      for (int j = ENDS ? 1 : 0; j < 3; ++j) d[b][j] = *(const gf32x4*)(dec + b * DD_BLOCK + 16 * j + 4 * q);
    tot = dec[DD_TOT];
#pragma unroll
    for (int j = DM_N - 1; j >= (ENDS ? DM_T0 : 0); --j) m[j] = mat<F32>(a.so, (p * a.H + h) * DM_N * MAT + j * MAT + mat_at<F32>(r16, 4 * q));
    if constexpr (HOLD) {
#pragma unroll
      for (int t = 0; t < NT; ++t) k[t] = oct<F32>(a.ko, col_at(p, t));
    }
  };
  if constexpr (ENDS) vo = Oct<F32>{};
  constexpr gf32x4 zero = {0.f, 0.f, 0.f, 0.f};
  // S[t]: rows 16 t + 4 q + r, column r16 of this wave's 16
  gf32x4 S[NT];
#pragma unroll
  for (int t = 0; t < NT; ++t) S[t] = zero;
  auto read = [&](gf32x4 (&x)[NT], const float* src) __attribute__((always_inline)) {
#pragma unroll
    for (int t = 0; t < NT; ++t)
#pragma unroll
      for (int r = 0; r < 4; ++r) x[t][r] = src[(size_t)(16 * t + r) * a.vp];
  };
  auto write = [&](float* dst) __attribute__((always_inline)) {
#pragma unroll
    for (int t = 0; t < NT; ++t)
#pragma unroll
      for (int r = 0; r < 4; ++r) dst[(size_t)(16 * t + r) * a.vp] = S[t][r];
  };
  auto first = [&]() __attribute__((always_inline)) {
    load_rows(sg.i0);
    load_rest(sg.i0);
  };
  if (ENDS || sg.n == 1) {
    first();
    if (seg == 0 && sq.pos0 > 0) read(S, st + ((sq.pos0 - 1) & 1) * half);
    if constexpr (ENDS) {
      if (seg == 0) write(seg_at(0));
      if (unit) {
#pragma unroll
        for (int t = 0; t < NT; ++t)
#pragma unroll
          for (int r = 0; r < 4; ++r) S[t][r] = 16 * t + 4 * q + r == col ? 1.f : 0.f;
      }
    }
  } else {
    // (the state itself may already be the new one: the copies are read)
    read(S, seg_at(min(seg, 1)));
    for (int j = 2; j <= seg; ++j) {  // the transition of segment j - 1 times what was, and what it added itself
      Tile<F32> s[NT];
#pragma unroll
      for (int t = 0; t < NT; ++t) s[t] = tile<F32>(S[t]);
      read(S, seg_at(j));
      const float* mt = mat_of(j) + r16 * NP + 4 * q;
#pragma unroll
      for (int t = 0; t < NT; ++t)
#pragma unroll
        for (int u = 0; u < NT; u += 2) {
          const Tile<F32> m0 = tile<F32>(*(const gf32x4*)(mt + 16 * t * NP + 16 * u)), m1 = tile<F32>(*(const gf32x4*)(mt + 16 * t * NP + 16 * u + 16));
          if constexpr (F32) {
            S[t] = mfma4(m1.f, s[u + 1].f, mfma4(m0.f, s[u].f, S[t]));
          } else {
            S[t] = mul(join(m0.h, m1.h), s[u], s[u + 1], S[t]);
            S[t] = mul8(join(m0.l, m1.l), join(s[u].h, s[u + 1].h), S[t]);
          }
        }
    }
    first();
  }
  for (int i = sg.i0; i < sg.i1; ++i) {
    gf32x4 c[2] = {zero, zero}, y[2] = {zero, zero};
#pragma unroll
    for (int t = 0; t < NT; t += 2) {
      const Tile<F32> s0 = tile<F32>(S[t]), s1 = tile<F32>(S[t + 1]);
#pragma unroll
      for (int b = 0; b < 2; ++b) {
        if constexpr (HOLD) {
          c[b] = mul(kr[b][t / 2], s0, s1, c[b]);
          if constexpr (!ENDS) y[b] = mul(x[b][t / 2], s0, s1, y[b]);
        } else {
          c[b] = mul(oct<F32>(a.kr, row_at(p0 + i, b, t)), s0, s1, c[b]);
          if constexpr (!ENDS) y[b] = mul(oct<F32>(a.qo, row_at(p0 + i, b, t)), s0, s1, y[b]);
        }
      }
    }
    __builtin_amdgcn_sched_barrier(0);
    load_rows(i + 1);
    __builtin_amdgcn_sched_barrier(0);
    gf32x4 v[2];  // in fp32: tokens 4 q + r, column r16
    if constexpr (F32) {
      v[0] = vo.a;
      v[1] = vo.b;
    } else {
#pragma unroll
      for (int b = 0; b < 2; ++b)
        v[b] = gf32x4{__uint_as_float(vo.u[2 * b] << 16), __uint_as_float(vo.u[2 * b] & 0xffff0000u),
                      __uint_as_float(vo.u[2 * b + 1] << 16), __uint_as_float(vo.u[2 * b + 1] & 0xffff0000u)};
    }
#pragma unroll
    for (int b = 0; b < 2; ++b) {
      v[b] -= d[b][2] * c[b];
      if constexpr (!ENDS) y[b] *= d[b][0];
    }
    const gf32x4 u0 = mul(m[DM_T0], tile<F32>(v[0]), zero);
    const Tile<F32> t0 = tile<F32>(u0);
    const gf32x4 u1 = mul(m[DM_T1], tile<F32>(mul(m[DM_L10], t0, v[1])), zero);
    const Tile<F32> t1 = tile<F32>(u1), e0 = tile<F32>(u0 * d[0][1]), e1 = tile<F32>(u1 * d[1][1]);
    if constexpr (!ENDS) {
      y[0] = mul(m[DM_A0], t0, y[0]);
      y[1] = mul(m[DM_A10], t0, y[1]);
      y[1] = mul(m[DM_A1], t1, y[1]);
    }
    // the state at the pair's end
#pragma unroll
    for (int t = 0; t < NT; ++t) S[t] = mul(HOLD ? k[HOLD ? t : 0] : oct<F32>(a.ko, col_at(p0 + i, t)), e0, e1, S[t] * tot);
    __builtin_amdgcn_sched_barrier(0);
    load_rest(i + 1);
    __builtin_amdgcn_sched_barrier(0);
    if (!ENDS && col < a.dv) {
#pragma unroll
      for (int b = 0; b < 2; ++b) {
        const int t = 32 * i + 16 * b + 4 * q;
        float* out = a.y + (size_t)(sq.row0 + t) * (a.H * a.dv) + h * a.dv + col;
#pragma unroll
        for (int r = 0; r < 4; ++r)
          if (t + r < sq.n) out[(size_t)r * a.H * a.dv] = y[b][r];
      }
    }
  }
  if constexpr (ENDS) {
    if (!unit) return write(seg_at(seg + 1));
    float* dst = mat_of(seg + 1) + 4 * q * NP + col;
#pragma unroll
    for (int t = 0; t < NT; ++t)
#pragma unroll
      for (int r = 0; r < 4; ++r) dst[(16 * t + r) * NP] = S[t][r];
  } else if (seg + 1 == sg.n) {
    write(st + ((sq.pos0 + sq.n - 1) & 1) * half);
  }
}

template <bool F32>
static void delta_walk(const LinScanArgs& a, hipStream_t st) {
  const int nscore = (a.n_chunks * a.H + 3) / 4, nkeep = (a.H * a.dv + 2 * a.G * a.N + 255) / 256;
  hipLaunchKernelGGL((delta_score_kernel<F32>), dim3(nscore + nkeep * a.n_seqs), dim3(256), 0, st, a, nscore, nkeep);
  auto walk = [&](auto nt) {
    constexpr int NT = decltype(nt)::value;
    const int n = a.H * (a.vp / 16), ne = n + a.H * NT;
    if (a.nseg > 1)
      hipLaunchKernelGGL((delta_walk_kernel<F32, NT, true>), dim3((ne + 7) / 8 * 8, a.n_seqs, a.nseg - 1), dim3(64), 0, st, a);
    hipLaunchKernelGGL((delta_walk_kernel<F32, NT, false>), dim3((n + 7) / 8 * 8, a.n_seqs, a.nseg), dim3(64), 0, st, a);
  };
  switch (a.np / 16) {
    case 2: walk(std::integral_constant<int, 2>{}); break;
    case 4: walk(std::integral_constant<int, 4>{}); break;
    case 6: walk(std::integral_constant<int, 6>{}); break;
    case 8: walk(std::integral_constant<int, 8>{}); break;
    case 12: walk(std::integral_constant<int, 12>{}); break;
    default: walk(std::integral_constant<int, 16>{}); break;
  }
}

// Two walks of 1 / n of the pairs, the first over the transition's columns too, instead of one of them all: from three on, where
// the chip has room
int delta_segments(int H, int np, int vp, int n_seqs, int blocks) {
  const int room = 4096 / std::max(1, H * (np + vp) / 16 * n_seqs);
  const int n = std::min({room, LIN_SEGS / std::max(1, n_seqs), blocks / (2 * DELTA_SEG_MIN), 8});
  return n < 3 ? 1 : n;
}

void launch_delta_walk(const LinScanArgs& a, hipStream_t st) { a.f32 ? delta_walk<true>(a, st) : delta_walk<false>(a, st); }

// ---- single tokens ----------------------------------------------------------------------------------
// With x = S^T k and w = S^T q of the state as it was: u = b (v - d x), o = d w + (k . q) u.  ROWS: rows of the
// state a thread asks for at once; a state of more (REREAD) is read a second time
template <bool F32, int ROWS, bool REREAD>
__global__ void __launch_bounds__(256) delta_step_kernel(LinScanArgs a) {
  extern __shared__ __attribute__((aligned(16))) float ls_smem[];
  __shared__ float red[4], dots[4][3];
  const int h = blockIdx.x, row = blockIdx.y, tid = threadIdx.x;
  const int pos = a.pos[row], slot = a.slot[row];
  const float* in = a.in + (size_t)row * a.ld;
  const int c4 = a.vp >> 2, nr = 256 / c4, col = 4 * (tid % c4), r0 = tid / c4;
  const bool mine = r0 < nr;
  float *sv = ls_smem, *sk = sv + a.vp, *sq = sk + a.np, *sx = sq + a.np, *sw = sx + nr * a.vp, *so = sw + nr * a.vp;
  const size_t hs = (size_t)a.np * a.vp, half = (size_t)a.slots * a.H * hs;
  float* st = a.state + ((size_t)slot * a.H + h) * hs;
  const float* src = st + ((pos - 1) & 1) * half;
  float* dst = st + (pos & 1) * half;
  float4 s[ROWS];
  auto fetch = [&](int n0) __attribute__((always_inline)) {
#pragma unroll
    for (int u = 0; u < ROWS; ++u) {
      const int n = n0 + u * nr;
      s[u] = make_float4(0.f, 0.f, 0.f, 0.f);
      if (pos > 0 && mine && n < a.np) s[u] = *(const float4*)(src + (size_t)n * a.vp + col);
    }
  };
  fetch(r0);  // (on its way while the operands are formed)
  const float dec = expf(-expf(a.a_log[h]) * lin_step_dt(a, in, h)), beta = 1.f / (1.f + expf(-in[a.b_off + h]));
  lin_step_conv<F32>(a, in, h, pos, slot, [&](int i, float u) { ls_smem[i] = u; });
  __syncthreads();
  float kk = 0.f, qq = 0.f, kq = 0.f;
  for (int n = tid; n < a.np; n += 256) {
    kk = fmaf(sk[n], sk[n], kk);
    qq = fmaf(sq[n], sq[n], qq);
    kq = fmaf(sk[n], sq[n], kq);
  }
#pragma unroll
  for (int d = 32; d; d >>= 1) {
    kk += __shfl_xor(kk, d, 64);
    qq += __shfl_xor(qq, d, 64);
    kq += __shfl_xor(kq, d, 64);
  }
  if ((tid & 63) == 0) {
    dots[tid >> 6][0] = kk;
    dots[tid >> 6][1] = qq;
    dots[tid >> 6][2] = kq;
  }
  float4 x = make_float4(0.f, 0.f, 0.f, 0.f), w = x;
  if (mine) {
    for (int n0 = r0; n0 < a.np; n0 += ROWS * nr) {
      if (REREAD && n0 != r0) fetch(n0);
#pragma unroll
      for (int u = 0; u < ROWS; ++u) {
        const int n = min(n0 + u * nr, a.np - 1);  // (past the end: the rows are zeros)
        const float k = sk[n], q = sq[n];
        x.x = fmaf(k, s[u].x, x.x); x.y = fmaf(k, s[u].y, x.y); x.z = fmaf(k, s[u].z, x.z); x.w = fmaf(k, s[u].w, x.w);
        w.x = fmaf(q, s[u].x, w.x); w.y = fmaf(q, s[u].y, w.y); w.z = fmaf(q, s[u].z, w.z); w.w = fmaf(q, s[u].w, w.w);
      }
    }
    *(float4*)(sx + r0 * a.vp + col) = x;
    *(float4*)(sw + r0 * a.vp + col) = w;
  }
  __syncthreads();
  kk = (dots[0][0] + dots[1][0]) + (dots[2][0] + dots[3][0]);
  qq = (dots[0][1] + dots[1][1]) + (dots[2][1] + dots[3][1]);
  kq = (dots[0][2] + dots[1][2]) + (dots[2][2] + dots[3][2]);
  const float ik = 1.f / sqrtf(kk + LIN_UNIT_EPS), iq = a.q_scale / sqrtf(qq + LIN_UNIT_EPS);
  if (mine) {
    x = make_float4(0.f, 0.f, 0.f, 0.f);
    for (int r = 0; r < nr; ++r) {
      const float4 p = *(const float4*)(sx + r * a.vp + col);
      x.x += p.x; x.y += p.y; x.z += p.z; x.w += p.w;
    }
    const float4 v = *(const float4*)(sv + col);
    const float f = -dec * ik, g = beta * ik;  // (the state takes k times ik)
    x.x = g * fmaf(f, x.x, v.x); x.y = g * fmaf(f, x.y, v.y); x.z = g * fmaf(f, x.z, v.z); x.w = g * fmaf(f, x.w, v.w);
    for (int n0 = r0; n0 < a.np; n0 += ROWS * nr) {
      if (REREAD) fetch(n0);
#pragma unroll
      for (int u = 0; u < ROWS; ++u) {
        const int n = n0 + u * nr;
        if (n >= a.np) break;
        const float k = sk[n];
        *(float4*)(dst + (size_t)n * a.vp + col) =
            make_float4(fmaf(k, x.x, dec * s[u].x), fmaf(k, x.y, dec * s[u].y), fmaf(k, x.z, dec * s[u].z), fmaf(k, x.w, dec * s[u].w));
      }
    }
    if (r0 == 0) {
      w = make_float4(0.f, 0.f, 0.f, 0.f);
      for (int r = 0; r < nr; ++r) {
        const float4 p = *(const float4*)(sw + r * a.vp + col);
        w.x += p.x; w.y += p.y; w.z += p.z; w.w += p.w;
      }
      const float c = iq * kq, d = iq * dec;
      *(float4*)(so + col) = make_float4(fmaf(c, x.x, d * w.x), fmaf(c, x.y, d * w.y), fmaf(c, x.z, d * w.z), fmaf(c, x.w, d * w.w));
    }
  }
  __syncthreads();
  float ss = 0.f;
  for (int j = tid; j < a.dv; j += 256) ss = fmaf(so[j], so[j], ss);
  lin_step_norm<F32>(a, in, h, row, so, ss, red);
}

template <bool F32>
static void delta_step(const LinScanArgs& a, hipStream_t st) {
  const int nr = 256 / (a.vp / 4), rows = (a.np + nr - 1) / nr;
  const size_t lds = (size_t)(2 * a.vp + 2 * a.np + 2 * nr * a.vp) * 4;
  const dim3 grid(a.H, a.n);
  if (rows <= 4) hipLaunchKernelGGL((delta_step_kernel<F32, 4, false>), grid, dim3(256), lds, st, a);
  else if (rows <= 16) hipLaunchKernelGGL((delta_step_kernel<F32, 16, false>), grid, dim3(256), lds, st, a);
  else hipLaunchKernelGGL((delta_step_kernel<F32, 16, true>), grid, dim3(256), lds, st, a);
}

void launch_delta_step(const LinScanArgs& a, hipStream_t st) { a.f32 ? delta_step<true>(a, st) : delta_step<false>(a, st); }

}  // namespace aios
