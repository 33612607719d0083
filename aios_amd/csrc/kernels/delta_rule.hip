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
//           leaves registers; other waves bring the operands through LDS, pairs ahead.
// Single tokens: delta_step, one workgroup per head and row, the norm included.
//
// fp32: state, decays, strengths, lengths, the system and its inverse, scores, norms, gates.  The products take bf16 operands:
// q, k, v as the convolution left them; the state, u and every matrix of the pair as two bf16 terms (hi + lo).  The 32-bit form
// (F32) runs the same steps on fp32 matrix instructions.
#include <algorithm>
#include <stdexcept>

#include "lds_dma.h"
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
// A workgroup's DELTA_W walkers take neighbouring columns of one head.  Its loaders bring what they read of a pair to LDS: 1 KB
// pieces, 16 bytes a lane in the order the products take them, pairs ahead.
constexpr int DELTA_W = 2, DELTA_L = 2;

template <bool F32, int NT>
struct DeltaStage {
  static constexpr int P = F32 ? 2 : 1;                                     // pieces of an Oct tile
  static constexpr int KR = 0, Q = KR + NT * P, K = Q + NT * P, M = K + NT * P, D = M + DM_N, V = D + 1;  // first pieces
  static constexpr int ALL = V + DELTA_W * P, EACH = (ALL + DELTA_L - 1) / DELTA_L;  // EACH: a loader requests
  static constexpr int BYTES = ALL * 1024;
  static constexpr int N = BYTES * 4 <= 150 * 1024 ? 4 : BYTES * 3 <= 150 * 1024 ? 3 : BYTES * 2 <= 150 * 1024 ? 2 : 1;
  static_assert(BYTES * N <= 150 * 1024, "LDS");
};

// loader l's part of pair p -> the stage at LDS address `to`
template <bool F32, int NT>
__device__ __forceinline__ void delta_request(const LinScanArgs& a, size_t p, int h, int vt0, int l, int lane, uint32_t to) {
  using L = DeltaStage<F32, NT>;
  constexpr int ES = F32 ? 4 : 2, ROWS = NT * 256 * ES, TILE = 512 * ES, R = NT / 2 * L::P;  // bytes of a block's rows, of an Oct tile
  const int nvt = a.vp >> 4, g = h / (a.H / a.G), r16 = lane & 15, q = lane >> 4;
  // a lane's 16 bytes of a piece: of an Oct tile or matrix (32 numbers a row), of an fp32 matrix
  const int by_oct = (r16 * 32 + 8 * q) * ES, by_mat = F32 ? (r16 * 16 + 4 * q) * 4 : by_oct;
  const uint8_t *kr = (const uint8_t*)a.kr + (2 * p * a.G + g) * ROWS, *qo = (const uint8_t*)a.qo + (2 * p * a.G + g) * ROWS;
  const uint8_t* ko = (const uint8_t*)a.ko + (p * a.G + g) * 2 * ROWS;
  const uint8_t* so = (const uint8_t*)a.so + (p * a.H + h) * DM_N * mat_size(F32) * ES;
  const uint8_t* vo = (const uint8_t*)a.vo + (p * a.H + h) * a.vp * 32 * ES;
#pragma unroll
  for (int j = 0; j < L::EACH; ++j) {
    const int u = min(l + DELTA_L * j, L::ALL - 1);  // (the last piece twice: the same bytes)
    const uint8_t* src;
    if (u < L::K) {
      const int r = u < L::Q ? u : u - L::Q, b = r >= R, t = r - b * R;
      src = (u < L::Q ? kr : qo) + (size_t)b * a.G * ROWS + (t / L::P) * TILE + (t % L::P) * 16 + by_oct;
    } else if (u < L::M) {
      src = ko + ((u - L::K) / L::P) * TILE + ((u - L::K) % L::P) * 16 + by_oct;
    } else if (u < L::D) {
      src = so + (u - L::M) * mat_size(F32) * ES + by_mat;
    } else if (u < L::V) {
      src = (const uint8_t*)(a.dec + (p * a.H + h) * DD_N) + (lane & 31) * 16;
    } else {
      src = vo + min(vt0 + (u - L::V) / L::P, nvt - 1) * TILE + ((u - L::V) % L::P) * 16 + by_oct;
    }
    pf_glds16(src, to + u * 1024);
  }
}

template <bool F32, int NT>
__global__ void __launch_bounds__(64 * (DELTA_W + DELTA_L)) __attribute__((amdgpu_waves_per_eu(!F32 && NT <= 8 ? 2 : 1)))
delta_walk_kernel(LinScanArgs a) {
  using L = DeltaStage<F32, NT>;
  // What a step reads is in registers before it begins where they and LDS have room (AHEAD): its rows since the step before was
  // half done, the rest since that one's end.
  constexpr bool AHEAD = L::N >= 3;
  extern __shared__ __attribute__((aligned(16))) uint8_t dw_smem[];
  const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const int nvt = a.vp >> 4, per_head = (nvt + DELTA_W - 1) / DELTA_W, groups = a.H * per_head;
  // (workgroups are dealt round-robin: a head's go to one XCD)
  const int w = (blockIdx.x & 7) * (gridDim.x >> 3) + (blockIdx.x >> 3);
  if (w >= groups) return;
  const int h = w / per_head, vt0 = (w - h * per_head) * DELTA_W;
  const ScanSeq sq = a.seqs[blockIdx.y];
  const int np = (sq.n + 2 * LIN_T - 1) / (2 * LIN_T), p0 = sq.b0 / 2;
  // Step i: the pieces it reads from LDS (its own, AHEAD the next one's) are there when all but the younger requests are; then one
  // barrier, after which nobody reads the stage any more that is filled next.
  if (wave >= DELTA_W) {
    const uint32_t lds0 = pf_lds_addr(dw_smem);
    auto request = [&](int i) __attribute__((always_inline)) {  // (past the end: the last one again)
      delta_request<F32, NT>(a, (size_t)(p0 + min(i, np - 1)), h, vt0, wave - DELTA_W, lane, lds0 + (uint32_t)(i % L::N) * L::BYTES);
    };
#pragma unroll
    for (int i = 0; i < (L::N > 1 ? L::N - 1 : 1); ++i) request(i);
    if constexpr (AHEAD) {
      pf_vmcnt<(L::N - 2) * L::EACH>();
      pf_barrier();
    }
    for (int i = 0; i < np; ++i) {
      pf_vmcnt<(AHEAD ? (L::N - 3) * L::EACH : 0)>();
      pf_barrier();
      if constexpr (L::N == 1) pf_barrier();
      request(i + (L::N > 1 ? L::N - 1 : 1));
    }
    pf_vmcnt<0>();  // (nothing may arrive in LDS that is another workgroup's by then)
    return;
  }
  const int r16 = lane & 15, q = lane >> 4;
  const bool mine = vt0 + wave < nvt;  // (a walker past the last column goes along)
  const int col = 16 * min(vt0 + wave, nvt - 1) + r16;
  const size_t hs = (size_t)a.np * a.vp, half = (size_t)a.slots * a.H * hs;
  float* st = a.state + ((size_t)sq.slot * a.H + h) * hs + (size_t)(4 * q) * a.vp + col;
  // S[t]: rows 16 t + 4 q + r, column r16 of this wave's 16
  constexpr gf32x4 zero = {0.f, 0.f, 0.f, 0.f};
  gf32x4 S[NT];
#pragma unroll
  for (int t = 0; t < NT; ++t) {
    S[t] = zero;
    if (sq.pos0 > 0) {
      const float* src = st + ((sq.pos0 - 1) & 1) * half + (size_t)(16 * t) * a.vp;
#pragma unroll
      for (int r = 0; r < 4; ++r) S[t][r] = src[(size_t)r * a.vp];
    }
  }
  Oct<F32> kr[2][AHEAD ? NT / 2 : 1], x[2][AHEAD ? NT / 2 : 1], k[AHEAD ? NT : 1], vo;
  Mat<F32> m[DM_N];
  gf32x4 d[2][3];
  float tot;
  auto stage = [&](int i) { return dw_smem + (i % L::N) * L::BYTES + lane * 16; };
  auto piece = [&](const uint8_t* sb, int u) __attribute__((always_inline)) {
    Oct<F32> o;
    if constexpr (F32) {
      o.a = *(const gf32x4*)(sb + u * 1024);
      o.b = *(const gf32x4*)(sb + (u + 1) * 1024);
    } else {
      o.u = *(const gu32x4*)(sb + u * 1024);
    }
    return o;
  };
  auto row = [&](int first, int b, int t) { return first + (b * NT + t) / 2 * L::P; };
  auto read_rows = [&](int i) __attribute__((always_inline)) {
    const uint8_t* sb = stage(i);
    if constexpr (AHEAD) {
#pragma unroll
      for (int t = 0; t < NT; t += 2)
#pragma unroll
        for (int b = 0; b < 2; ++b) {
          kr[b][t / 2] = piece(sb, row(L::KR, b, t));
          x[b][t / 2] = piece(sb, row(L::Q, b, t));
        }
    }
  };
  auto read_rest = [&](int i) __attribute__((always_inline)) {
    const uint8_t* sb = stage(i);
    const float* dec = (const float*)(sb - lane * 16 + L::D * 1024);
    vo = piece(sb, L::V + wave * L::P);
#pragma unroll
    for (int b = 0; b < 2; ++b)
#pragma unroll
      for (int j = 0; j < 3; ++j) d[b][j] = *(const gf32x4*)(dec + b * DD_BLOCK + 16 * j + 4 * q);
    tot = dec[DD_TOT];
#pragma unroll
    for (int j = DM_N - 1; j >= 0; --j) {
      if constexpr (F32) m[j].f = *(const gf32x4*)(sb + (L::M + j) * 1024);
      else m[j].u = *(const gu32x4*)(sb + (L::M + j) * 1024);
    }
    if constexpr (AHEAD) {
#pragma unroll
      for (int t = 0; t < NT; ++t) k[t] = piece(sb, L::K + t * L::P);
    }
  };
  if constexpr (AHEAD) {
    pf_barrier();
    read_rows(0);
    read_rest(0);
  }
  for (int i = 0; i < np; ++i) {
    __builtin_amdgcn_sched_barrier(0);
    // (without AHEAD the last step's reads may not have come back yet)
    if constexpr (!AHEAD) asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
    pf_barrier();
    const uint8_t* sb = stage(i);
    if constexpr (!AHEAD) read_rest(i);
    gf32x4 c[2] = {zero, zero}, y[2] = {zero, zero};
#pragma unroll
    for (int t = 0; t < NT; t += 2) {
      const Tile<F32> s0 = tile<F32>(S[t]), s1 = tile<F32>(S[t + 1]);
#pragma unroll
      for (int b = 0; b < 2; ++b) {
        c[b] = mul(AHEAD ? kr[b][AHEAD ? t / 2 : 0] : piece(sb, row(L::KR, b, t)), s0, s1, c[b]);
        y[b] = mul(AHEAD ? x[b][AHEAD ? t / 2 : 0] : piece(sb, row(L::Q, b, t)), s0, s1, y[b]);
      }
    }
    if constexpr (AHEAD) {
      __builtin_amdgcn_sched_barrier(0);
      read_rows(i + 1);
      __builtin_amdgcn_sched_barrier(0);
    }
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
      y[b] *= d[b][0];
    }
    const gf32x4 u0 = mul(m[DM_T0], tile<F32>(v[0]), zero);
    const Tile<F32> t0 = tile<F32>(u0);
    const gf32x4 u1 = mul(m[DM_T1], tile<F32>(mul(m[DM_L10], t0, v[1])), zero);
    const Tile<F32> t1 = tile<F32>(u1), e0 = tile<F32>(u0 * d[0][1]), e1 = tile<F32>(u1 * d[1][1]);
    // the state at the pair's end
#pragma unroll
    for (int t = 0; t < NT; ++t) S[t] = mul(AHEAD ? k[AHEAD ? t : 0] : piece(sb, L::K + t * L::P), e0, e1, S[t] * tot);
    y[0] = mul(m[DM_A0], t0, y[0]);
    y[1] = mul(m[DM_A10], t0, y[1]);
    y[1] = mul(m[DM_A1], t1, y[1]);
    if constexpr (AHEAD) {
      __builtin_amdgcn_sched_barrier(0);
      read_rest(i + 1);
      __builtin_amdgcn_sched_barrier(0);
    }
    if (mine && col < a.dv) {
#pragma unroll
      for (int b = 0; b < 2; ++b) {
        const int t = 32 * i + 16 * b + 4 * q;
        float* out = a.y + (size_t)(sq.row0 + t) * (a.H * a.dv) + h * a.dv + col;
#pragma unroll
        for (int r = 0; r < 4; ++r)
          if (t + r < sq.n) out[(size_t)r * a.H * a.dv] = y[b][r];
      }
    }
    if constexpr (L::N == 1) {
      asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory");
      pf_barrier();
    }
  }
  if (!mine) return;
  float* dst = st + ((sq.pos0 + sq.n - 1) & 1) * half;
#pragma unroll
  for (int t = 0; t < NT; ++t)
#pragma unroll
    for (int r = 0; r < 4; ++r) dst[(size_t)(16 * t + r) * a.vp] = S[t][r];
}

template <bool F32>
static void delta_walk(const LinScanArgs& a, hipStream_t st) {
  const int nscore = (a.n_chunks * a.H + 3) / 4, nkeep = (a.H * a.dv + 2 * a.G * a.N + 255) / 256;
  hipLaunchKernelGGL((delta_score_kernel<F32>), dim3(nscore + nkeep * a.n_seqs), dim3(256), 0, st, a, nscore, nkeep);
  auto walk = [&](auto nt) {
    constexpr int NT = decltype(nt)::value;
    using L = DeltaStage<F32, NT>;
    const int groups = a.H * ((a.vp / 16 + DELTA_W - 1) / DELTA_W);
    hipLaunchKernelGGL((delta_walk_kernel<F32, NT>), dim3((groups + 7) / 8 * 8, a.n_seqs), dim3(64 * (DELTA_W + DELTA_L)),
                       L::N * L::BYTES, st, a);
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
