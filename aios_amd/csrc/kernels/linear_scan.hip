// Linear recurrences with a matrix state (mixers.h LinScanArgs): per head S_t = d_t S_{t-1} + k_t v_t^T, o_t = S_t^T q_t.
//
// Portions, in blocks of 16 tokens:
//   conv (LIN_HEAD)    a thread per channel and block: convolution, SiLU, operands in the order the walk reads them
//   prep / score       decays, and the block's own scores A[t][s] = q_t . (d_t .. d_{s+1} k_s), s <= t
//   walk               a wave owns a head and 16 columns of v: S [N][16] stays in its accumulators from block to block,
//                        o = (q with the decay since the block's start) S + A v,
//                        S = (decay of the block) S + (k with the decay to the block's end)^T v.
//                      A 16 x 16 accumulator tile is, lane for lane, the second operand of the 16-deep product, so S never
//                      leaves registers and the waves need no barrier.  Operands are requested several blocks ahead.
//                      Where heads and columns leave compute units idle, a portion is walked in segments side by side: a
//                      first walk takes every segment but the last from zero (the first one from the state) to its end,
//                      without outputs; the second starts each segment from what those before it make together.
//   norm               root-mean-square of the parts, weight, output gate
// LIN_DELTA has a score and a walk of its own (delta_rule.hip); convolution and norm are shared.
// Single tokens: lin_step, one workgroup per head and row (convolution, decays, state and, for LIN_KEY, the norm).
//
// fp32: state, decays, step sizes, cumulative decays, scores, norms, gates.  The products take bf16 operands: q, k, v and
// the convolution's outputs as they are, everything that carries a decay or comes from the state as two bf16 terms
// (hi + lo).  The 32-bit form (F32) runs the same steps on fp32 matrix instructions.
#include <algorithm>
#include <stdexcept>

#include "lin_common.h"

namespace aios {

int lin_pad_n(int n) {
  for (int t : {32, 64, 96, 128, 192, 256})
    if (n <= t) return t;
  return 0;
}

// numbers per block of LIN_T tokens; bf16: decayed operands have a second plane behind the first
LinWs lin_ws(int kind, int H, int G, int np, int vp, bool f32) {
  const size_t g = kind == LIN_KEY ? H : G, two = f32 ? 1 : 2, q = g * np * LIN_T;
  LinWs w;
  w.qo = kind == LIN_KEY ? q * two : q;
  w.ko = w.qo;
  w.kr = kind != LIN_KEY ? q : 0;
  w.vo = (size_t)H * vp * LIN_T;
  w.so = (size_t)H * 256 * two * (kind == LIN_DELTA ? 3 : 1);
  w.dec = kind == LIN_KEY ? (size_t)H * np : (size_t)H * (kind == LIN_DELTA ? 64 : 48);
  return w;
}

// ---- LIN_HEAD, LIN_DELTA: convolution --------------------------------------------------------------------------
constexpr int LC_T = 128;

// TM: taps at most; PAIRS: a pair of blocks, in the operands' order of delta_rule.hip
template <bool F32, int TM, bool PAIRS>
__global__ void __launch_bounds__(LC_T) lin_conv_kernel(LinScanArgs a) {
  constexpr int TOK = PAIRS ? 2 * LIN_T : LIN_T;
  LinBlock bl = lin_block(a, PAIRS ? 2 * blockIdx.y : blockIdx.y);
  if (bl.n < 1) return;
  if (PAIRS) bl.n = a.chunks[blockIdx.y].n;
  const int nx = a.H * a.vp, ng = a.G * a.np;
  int c = blockIdx.x * LC_T + threadIdx.x;
  if (c >= nx + 2 * ng) return;
  // which input column
  const int C = a.H * a.dv + 2 * a.G * a.N;
  int sec = 0, hd, i, raw = -1;
  if (c < nx) {
    hd = c / a.vp;
    i = c - hd * a.vp;
    if (i < a.dv) raw = hd * a.dv + i;
  } else {
    sec = 1 + (c - nx) / ng;
    const int k = (c - nx) % ng;
    hd = k / a.np;
    i = k - hd * a.np;
    if (i < a.N) raw = a.H * a.dv + (sec - 1) * a.G * a.N + hd * a.N + i;
  }
  float u[TOK];
#pragma unroll
  for (int t = 0; t < TOK; ++t) u[t] = 0.f;
  if (raw >= 0) {
    float w[TM], x[TOK + TM - 1];  // w[d]: tap of lag d
#pragma unroll
    for (int d = 0; d < TM; ++d) w[d] = d < a.taps ? a.conv_w[(size_t)raw * a.taps + a.taps - 1 - d] : 0.f;
#pragma unroll
    for (int j = 0; j < TOK + TM - 1; ++j) {
      const int t = j - (TM - 1), p = bl.pos0 + t;  // token t of the block
      x[j] = 0.f;
      if (t >= bl.n || -t >= a.taps) continue;
      if (p >= bl.seq_pos0) x[j] = a.in[(size_t)(bl.row0 + t) * a.ld + a.x_off + raw];
      else if (p >= 0) x[j] = a.ring[((size_t)bl.slot * a.taps + p % a.taps) * C + raw];
    }
    const float b = a.conv_b ? a.conv_b[raw] : 0.f;
#pragma unroll
    for (int t = 0; t < TOK; ++t) {
      float s = b;
#pragma unroll
      for (int d = 0; d < TM; ++d) s = fmaf(w[d], x[t + TM - 1 - d], s);
      u[t] = t < bl.n ? ls_silu<F32>(s) : 0.f;
    }
  }
  const size_t blk = blockIdx.y;
  if constexpr (PAIRS) {
    if (sec < 2) {  // (four tokens of the first block, then the same of the second)
      float o[2][16];
#pragma unroll
      for (int t = 0; t < TOK; ++t) o[(t & 15) >> 3][((t >> 2) & 1) * 8 + (t >> 4) * 4 + (t & 3)] = u[t];
      void* cols = sec == 0 ? a.vo : a.ko;
      const size_t at = (sec == 0 ? (blk * a.H + hd) * a.vp + i : (blk * a.G + hd) * a.np + i) * TOK;
      put16<F32>(cols, at, o[0]);
      put16<F32>(cols, at + 16, o[1]);
      if (sec == 0) return;
    }
#pragma unroll
    for (int t = 0; t < TOK; ++t)
      put1<F32>(sec == 1 ? a.kr : a.qo, ((2 * blk + (t >> 4)) * a.G + hd) * a.np * 16 + pair_row(i, t & 15), u[t]);
  } else {
    if (sec == 0) return put16<F32>(a.vo, ((blk * a.H + hd) * a.vp + i) * 16, u);
    const size_t base = (blk * a.G + hd) * a.np;
    if (sec == 1) put16<F32>(a.ko, (base + i) * 16, u);
    void* rows = sec == 1 ? a.kr : a.qo;
#pragma unroll
    for (int t = 0; t < 16; ++t) put1<F32>(rows, (base + (i & ~15)) * 16 + t * 16 + (i & 15), u[t]);
  }
}

// ---- LIN_HEAD: decays and scores; the last inputs into the ring -----------------------------------------
template <bool F32>
__global__ void __launch_bounds__(256) lin_score_kernel(LinScanArgs a, int nscore, int nkeep) {
  if ((int)blockIdx.x >= nscore) return lin_keep(a, blockIdx.x - nscore, nkeep);
  const int lane = threadIdx.x & 63, idx = blockIdx.x * 4 + (threadIdx.x >> 6);
  const int blk = idx / a.H, h = idx - blk * a.H;
  if (blk >= 2 * a.n_chunks) return;
  const LinBlock bl = lin_block(a, blk);
  if (bl.n < 1) return;
  const int r16 = lane & 15, q = lane >> 4;
  // token r16: step size, log decay, its running sum
  const float e = expf(a.a_log[h]);
  float dt = 0.f;
  if (r16 < bl.n) dt = ls_softplus(a.in[(size_t)(bl.row0 + r16) * a.ld + a.dt_off + h] + a.dt_b[h]);
  float cum = -e * dt;
#pragma unroll
  for (int d = 1; d < 16; d <<= 1) {
    const float o = __shfl_up(cum, d, 16);
    if (r16 >= d) cum += o;
  }
  const float tot = __shfl(cum, 15, 16);
  float* dec = a.dec + ((size_t)blk * a.H + h) * 48;
  if (q == 0) {
    dec[r16] = expf(cum);
    dec[16 + r16] = dt * expf(tot - cum);
    if (r16 == 0) dec[32] = expf(tot);
  }
  // A^T[s][t] = k_s . q_t: a lane holds s = 4 q + r, t = r16
  const size_t base = ((size_t)blk * a.G + h / (a.H / a.G)) * a.np * 16 + r16 * 16 + 4 * q;
  gf32x4 acc = {0.f, 0.f, 0.f, 0.f};
  for (int i = 0; i < a.np / 16; i += 2) {
    const size_t at = base + (size_t)i * 256;
    if constexpr (F32) {
      acc = mfma4(*(const gf32x4*)((const float*)a.kr + at), *(const gf32x4*)((const float*)a.qo + at), acc);
      acc = mfma4(*(const gf32x4*)((const float*)a.kr + at + 256), *(const gf32x4*)((const float*)a.qo + at + 256), acc);
    } else {
      const bf16_t *kr = (const bf16_t*)a.kr + at, *qr = (const bf16_t*)a.qo + at;
      acc = mfma32(*(const lu2*)kr, *(const lu2*)(kr + 256), *(const lu2*)qr, *(const lu2*)(qr + 256), acc);
    }
  }
#pragma unroll
  for (int r = 0; r < 4; ++r) {
    const int s = 4 * q + r;
    const float cs = __shfl(cum, s, 16), ds = __shfl(dt, s, 16);
    acc[r] = s <= r16 ? acc[r] * ds * expf(cum - cs) : 0.f;
  }
  const size_t at = ((size_t)blk * a.H + h) * (F32 ? 256 : 512) + r16 * 16 + 4 * q;
  if constexpr (F32) {
    *(gf32x4*)((float*)a.so + at) = acc;
  } else {
    lu2 hi, lo;
    split4(acc, hi, lo);
    *(lu2*)((bf16_t*)a.so + at) = hi;
    *(lu2*)((bf16_t*)a.so + at + 256) = lo;
  }
}

// ---- LIN_KEY: decays, operands and scores of one (block, head) ---------------------------------------------
__device__ __forceinline__ float row16_sum(float v) {  // over 16 neighbouring lanes
  v += __uint_as_float(__builtin_amdgcn_update_dpp(0, __float_as_uint(v), 0xB1, 0xf, 0xf, true));
  v += __uint_as_float(__builtin_amdgcn_update_dpp(0, __float_as_uint(v), 0x4E, 0xf, 0xf, true));
  v += __uint_as_float(__builtin_amdgcn_update_dpp(0, __float_as_uint(v), 0x141, 0xf, 0xf, true));
  v += __uint_as_float(__builtin_amdgcn_update_dpp(0, __float_as_uint(v), 0x140, 0xf, 0xf, true));
  return v;
}

template <bool F32, int NT>
__global__ void __launch_bounds__(256) lin_key_prep_kernel(LinScanArgs a) {
  constexpr int NP = 16 * NT;
  extern __shared__ __attribute__((aligned(16))) float lk_smem[];
  float *sd = lk_smem, *sq = sd + 16 * NP, *sk = sq + 16 * NP, *sa = sk + 16 * NP;
  const int h = blockIdx.x, tid = threadIdx.x;
  const size_t blk = blockIdx.y;
  const LinBlock bl = lin_block(a, blk);
  if (bl.n < 1) return;
  const float* in = a.in + (size_t)bl.row0 * a.ld;
  for (int i = tid; i < 16 * a.rank; i += 256) {
    const int t = i / a.rank;
    sa[i] = t < bl.n ? in[(size_t)t * a.ld + a.a_off + i - t * a.rank] : 0.f;
  }
  for (int j = tid; j < a.vp; j += 256) {
    float v[16];
#pragma unroll
    for (int t = 0; t < 16; ++t) v[t] = t < bl.n && j < a.dv ? in[(size_t)t * a.ld + a.v_off + h * a.dv + j] : 0.f;
    put16<F32>(a.vo, ((blk * a.H + h) * a.vp + j) * 16, v);
  }
  __syncthreads();
  // log decays: a thread owns TG tokens of a channel
  constexpr int GR = NP <= 32 ? 8 : NP <= 64 ? 4 : NP <= 128 ? 2 : 1, TG = 16 / GR;
  if (tid < GR * NP) {
    const int n = tid % NP, t0 = tid / NP * TG;
    const bool real = n < a.N;
    const int c = h * a.N + (real ? n : 0);
    float z[TG], qv[TG], kv[TG];
#pragma unroll
    for (int t = 0; t < TG; ++t) {
      const bool ok = real && t0 + t < bl.n;
      qv[t] = ok ? in[(size_t)(t0 + t) * a.ld + a.q_off + c] : 0.f;
      kv[t] = ok ? in[(size_t)(t0 + t) * a.ld + a.k_off + c] : 0.f;
      z[t] = a.a2_b[c];
    }
    const float *w = a.a2 + (size_t)c * a.rank, *ar = sa + t0 * a.rank;
    int r = 0;
    for (; r + 4 <= a.rank; r += 4) {
      const float w0 = w[r], w1 = w[r + 1], w2 = w[r + 2], w3 = w[r + 3];
#pragma unroll
      for (int t = 0; t < TG; ++t) {
        const float* x = ar + t * a.rank + r;
        z[t] = fmaf(w3, x[3], fmaf(w2, x[2], fmaf(w1, x[1], fmaf(w0, x[0], z[t]))));
      }
    }
    for (; r < a.rank; ++r)
#pragma unroll
      for (int t = 0; t < TG; ++t) z[t] = fmaf(w[r], ar[t * a.rank + r], z[t]);
#pragma unroll
    for (int t = 0; t < TG; ++t) {
      const int i = (t0 + t) * NP + n;
      sd[i] = real && t0 + t < bl.n ? -ls_softplus(-z[t]) * a.inv_tau : 0.f;
      sq[i] = qv[t] * a.q_scale;
      sk[i] = kv[t];
    }
  }
  __syncthreads();
  const size_t base = (blk * a.H + h) * NP, plane = (size_t)2 * a.n_chunks * a.H * NP * 16;
  if (tid < NP) {
    const int n = tid;
    float cum[16], s = 0.f, k[16];
#pragma unroll
    for (int t = 0; t < 16; ++t) cum[t] = s += sd[t * NP + n];
    a.dec[base + n] = expf(s);
    const size_t at = (base + (n & ~15)) * 16 + (n & 15);
#pragma unroll
    for (int t = 0; t < 16; ++t) {
      const float qd = sq[t * NP + n] * expf(cum[t]);
      k[t] = sk[t * NP + n] * expf(s - cum[t]);
      put1<F32>(a.qo, at + t * 16, qd);
      if constexpr (!F32) put1<F32>(a.qo, plane + at + t * 16, qd - bf16_to_f32(f32_to_bf16(qd)));
    }
    put16<F32>(a.ko, (base + n) * 16, k);
    if constexpr (!F32) {
#pragma unroll
      for (int t = 0; t < 16; ++t) k[t] -= bf16_to_f32(f32_to_bf16(k[t]));
      put16<F32>(a.ko, plane + (base + n) * 16, k);
    }
  }
  __syncthreads();
  for (int i = tid; i < 16 * NP; i += 256) sd[i] = expf(sd[i]);
  __syncthreads();
  // A[t][s]: 16 lanes share s and walk t; lane p carries k_s decayed to t at columns p + 16 i
  const int s = tid >> 4, p = tid & 15;
  float w[NT], mine = 0.f;
#pragma unroll
  for (int i = 0; i < NT; ++i) w[i] = 0.f;
#pragma unroll
  for (int t = 0; t < 16; ++t) {
    float acc = 0.f;
#pragma unroll
    for (int i = 0; i < NT; ++i) {
      const int at = t * NP + p + 16 * i;
      w[i] = t == s ? sk[at] : w[i] * sd[at];
      acc = fmaf(sq[at], w[i], acc);
    }
    acc = row16_sum(acc);
    if (p == t) mine = acc;
  }
  const size_t at = (blk * a.H + h) * (F32 ? 256 : 512) + p * 16 + s;
  put1<F32>(a.so, at, mine);
  if constexpr (!F32) put1<F32>(a.so, at + 256, mine - bf16_to_f32(f32_to_bf16(mine)));
}

// ---- the walk ---------------------------------------------------------------------------------------
template <bool F32, bool KEY, int NT>
struct LinOps;
template <bool KEY, int NT>
struct LinOps<false, KEY, NT> {
  lu2 q[NT], ql[KEY ? NT : 1], k[NT], kl[KEY ? NT : 1], s, sl, v;
  gf32x4 d[KEY ? NT : 2];
  float tot;
};
template <bool KEY, int NT>
struct LinOps<true, KEY, NT> {
  gf32x4 q[NT], k[NT], s, v, d[KEY ? NT : 2];
  float tot;
};

// buffers of operands in registers: requests run that many blocks ahead, less one
template <bool F32, bool KEY, int NT>
constexpr int lin_depth() {
  if (F32) return 2;
  return KEY ? (NT <= 2 ? 4 : NT <= 4 ? 3 : NT <= 6 ? 4 : NT <= 8 ? 3 : 2) : (NT <= 4 ? 4 : NT <= 6 ? 3 : NT <= 8 ? 2 : NT <= 12 ? 3 : 2);
}
// waves a SIMD whose registers fit
constexpr int lin_waves(bool key, int nt) { return nt <= (key ? 4 : 8) ? 2 : 1; }

// the blocks of a portion that a segment walks: [i0, i1), and how many segments there are
struct LinSeg {
  int i0, i1, n;
};
__device__ __forceinline__ LinSeg lin_seg(int nb, int nseg, int seg) {
  const int per = max(LIN_SEG_MIN, (nb + nseg - 1) / nseg);
  return LinSeg{seg * per, min(nb, (seg + 1) * per), (nb + per - 1) / per};
}

// ENDS: the first walk of a portion in segments (no outputs; segment s leaves what it ends with at seg[s + 1], its decay
// at seg_dec[s + 1]; the first one also copies the state it starts from to seg[0])
template <bool F32, bool KEY, int NT, bool ENDS>
__global__ void __launch_bounds__(256) __attribute__((amdgpu_waves_per_eu(F32 ? 1 : lin_waves(KEY, NT)))) lin_walk_kernel(LinScanArgs a) {
  constexpr int NP = 16 * NT, DEPTH = lin_depth<F32, KEY, NT>();
  using T = std::conditional_t<F32, float, bf16_t>;
  using V = std::conditional_t<F32, gf32x4, lu2>;
  const int lane = threadIdx.x & 63, nvt = a.vp >> 4;
  const int w = __builtin_amdgcn_readfirstlane(blockIdx.x * 4 + (threadIdx.x >> 6));
  if (w >= a.H * nvt) return;
  const int h = w / nvt, vt = w - h * nvt, g = KEY ? h : h / (a.H / a.G), ng = KEY ? a.H : a.G;
  const int r16 = lane & 15, q = lane >> 4;
  const ScanSeq sq = a.seqs[blockIdx.y];
  const int nb = (sq.n + LIN_T - 1) / LIN_T, col = 16 * vt + r16, seg = blockIdx.z;
  const LinSeg sg = lin_seg(nb, a.nseg, seg);
  if (seg >= sg.n) return;
  const size_t hs = (size_t)a.np * a.vp, half = (size_t)a.slots * a.H * hs;
  const size_t at = (size_t)(4 * q) * a.vp + col;  // of this lane in a head's state
  float* st = a.state + ((size_t)sq.slot * a.H + h) * hs + at;
  // segment j of this portion and head
  auto seg_at = [&](int j) { return a.seg + (((size_t)blockIdx.y * a.nseg + j) * a.H + h) * hs + at; };
  auto dec_at = [&](int j) { return a.seg_dec + (((size_t)blockIdx.y * a.nseg + j) * a.H + h) * a.np; };
  const size_t plane = (size_t)2 * a.n_chunks * a.H * NP * 16;
  using Ops = LinOps<F32, KEY, NT>;
  auto load = [&](Ops& o, int i) __attribute__((always_inline)) {
    const size_t b = sq.b0 + min(i, sg.i1 - 1);  // (past the end: re-reads)
    const T* qo = (const T*)a.qo + (b * ng + g) * NP * 16 + r16 * 16 + 4 * q;
    const T* ko = (const T*)a.ko + (b * ng + g) * NP * 16 + r16 * 16 + 4 * q;
#pragma unroll
    for (int t = 0; t < NT; ++t) {
      o.k[t] = *(const V*)(ko + 256 * t);
      if constexpr (KEY && !F32) o.kl[t] = *(const V*)(ko + plane + 256 * t);
      if constexpr (ENDS) continue;
      o.q[t] = *(const V*)(qo + 256 * t);
      if constexpr (KEY && !F32) o.ql[t] = *(const V*)(qo + plane + 256 * t);
    }
    const T* so = (const T*)a.so + (b * a.H + h) * (F32 ? 256 : 512) + r16 * 16 + 4 * q;
    if constexpr (!ENDS) {
      o.s = *(const V*)so;
      if constexpr (!F32) o.sl = *(const V*)(so + 256);
    }
    o.v = *(const V*)((const T*)a.vo + ((b * a.H + h) * a.vp + col) * 16 + 4 * q);
    if constexpr (KEY) {
#pragma unroll
      for (int t = 0; t < NT; ++t) o.d[t] = *(const gf32x4*)(a.dec + (b * a.H + h) * NP + 16 * t + 4 * q);
    } else {
      const float* d = a.dec + (b * a.H + h) * 48;
      if constexpr (!ENDS) o.d[0] = *(const gf32x4*)(d + 4 * q);
      o.d[1] = *(const gf32x4*)(d + 16 + 4 * q);
      o.tot = d[32];
    }
  };
  Ops o[DEPTH];
  static_for<DEPTH - 1>([&](auto d) { load(o[d], sg.i0 + d); });
  // S[t]: rows 16 t + 4 q + r, column r16 of this wave's 16
  gf32x4 S[NT];
  auto read = [&](gf32x4 (&x)[NT], const float* src) __attribute__((always_inline)) {
#pragma unroll
    for (int t = 0; t < NT; ++t)
#pragma unroll
      for (int r = 0; r < 4; ++r) x[t][r] = src[(size_t)(16 * t + r) * a.vp];
  };
  auto write = [&](float* dst) {
#pragma unroll
    for (int t = 0; t < NT; ++t)
#pragma unroll
      for (int r = 0; r < 4; ++r) dst[(size_t)(16 * t + r) * a.vp] = S[t][r];
  };
  if (ENDS || a.nseg == 1 || sg.n == 1) {
    if (sq.pos0 > 0 && seg == 0) {
      read(S, st + ((sq.pos0 - 1) & 1) * half);
    } else {
#pragma unroll
      for (int t = 0; t < NT; ++t) S[t] = gf32x4{0.f, 0.f, 0.f, 0.f};
    }
    if constexpr (ENDS) {
      if (seg == 0) write(seg_at(0));
      if (seg + 1 >= sg.n) return;  // (the last one's end is the second walk's)
    }
  } else {
    // (the state itself may already be the new one: the copies are read)
    read(S, seg_at(min(seg, 1)));
    for (int j = 2; j <= seg; ++j) {
      gf32x4 e[NT];
      read(e, seg_at(j));
      const float* d = dec_at(j);
#pragma unroll
      for (int t = 0; t < NT; ++t) S[t] = S[t] * *(const gf32x4*)(d + 16 * t + 4 * q) + e[t];
    }
  }
  gf32x4 D[ENDS && KEY ? NT : 1];  // decay of the segment
  if constexpr (ENDS) {
#pragma unroll
    for (int t = 0; t < (KEY ? NT : 1); ++t) D[t] = gf32x4{1.f, 1.f, 1.f, 1.f};
  }
  const float skip = KEY || ENDS ? 0.f : a.D[h];
  auto step = [&](const Ops& o, int i) __attribute__((always_inline)) {
    gf32x4 y0 = {0.f, 0.f, 0.f, 0.f}, y1 = y0;
    gf32x4 vf;  // v in fp32: tokens 4 q + r, column r16
    if constexpr (F32) vf = o.v;
    else
      vf = gf32x4{__uint_as_float(o.v.x << 16), __uint_as_float(o.v.x & 0xffff0000u), __uint_as_float(o.v.y << 16),
                  __uint_as_float(o.v.y & 0xffff0000u)};
    if constexpr (ENDS) {
    } else if constexpr (F32) {
#pragma unroll
      for (int t = 0; t < NT; t += 2) {
        y0 = mfma4(o.q[t], S[t], y0);
        y1 = mfma4(o.q[t + 1], S[t + 1], y1);
      }
      y0 += y1;
      if constexpr (!KEY) y0 *= o.d[0];
      y0 = mfma4(o.s, o.v, y0);
    } else {
#pragma unroll
      for (int t = 0; t < NT; t += 2) {
        lu2 h0, l0, h1, l1;
        split4(S[t], h0, l0);
        split4(S[t + 1], h1, l1);
        y0 = mfma32(o.q[t], o.q[t + 1], h0, h1, y0);
        y1 = mfma32(o.q[t], o.q[t + 1], l0, l1, y1);
        if constexpr (KEY) y1 = mfma32(o.ql[t], o.ql[t + 1], h0, h1, y1);
      }
      y0 += y1;
      if constexpr (!KEY) y0 *= o.d[0];
      y0 = mfma32(o.s, o.sl, o.v, o.v, y0);
    }
    if constexpr (!KEY && !ENDS) y0 += skip * vf;
    // the state at the block's end
    if constexpr (KEY) {
#pragma unroll
      for (int t = 0; t < NT; ++t) {
        S[t] *= o.d[t];
        if constexpr (ENDS) D[t] *= o.d[t];
        if constexpr (F32) S[t] = mfma4(o.k[t], o.v, S[t]);
        else S[t] = mfma32(o.k[t], o.kl[t], o.v, o.v, S[t]);
      }
    } else {
      if constexpr (ENDS) D[0] *= o.tot;
      const gf32x4 vd = vf * o.d[1];
      lu2 vh, vl;
      if constexpr (!F32) split4(vd, vh, vl);
#pragma unroll
      for (int t = 0; t < NT; ++t) {
        S[t] *= o.tot;
        if constexpr (F32) S[t] = mfma4(o.k[t], vd, S[t]);
        else S[t] = mfma32(o.k[t], o.k[t], vh, vl, S[t]);
      }
    }
    if (!ENDS && col < a.dv) {
      float* y = a.y + (size_t)(sq.row0 + 16 * i + 4 * q) * (a.H * a.dv) + h * a.dv + col;
      if (16 * i + 16 <= sq.n) {
#pragma unroll
        for (int r = 0; r < 4; ++r) y[(size_t)r * a.H * a.dv] = y0[r];
      } else {
#pragma unroll
        for (int r = 0; r < 4; ++r)
          if (16 * i + 4 * q + r < sq.n) y[(size_t)r * a.H * a.dv] = y0[r];
      }
    }
  };
  int i = sg.i0;
  for (; i + DEPTH <= sg.i1; i += DEPTH)
    static_for<DEPTH>([&](auto d) __attribute__((always_inline)) {
      load(o[(d + DEPTH - 1) % DEPTH], i + d + DEPTH - 1);
      step(o[d], i + d);
    });
  static_for<DEPTH - 1>([&](auto d) __attribute__((always_inline)) {
    if (i + d < sg.i1) step(o[d], i + d);
  });
  if constexpr (ENDS) {
    write(seg_at(seg + 1));
    if (vt == 0 && r16 == 0) {
#pragma unroll
      for (int t = 0; t < NT; ++t) *(gf32x4*)(dec_at(seg + 1) + 16 * t + 4 * q) = D[KEY ? t : 0];
    }
  } else if (seg + 1 == sg.n) {
    write(st + ((sq.pos0 + sq.n - 1) & 1) * half);
  }
}

// ---- single tokens ----------------------------------------------------------------------------------
template <bool F32, bool KEY>
__global__ void __launch_bounds__(256) lin_step_kernel(LinScanArgs a) {
  extern __shared__ __attribute__((aligned(16))) float ls_smem[];
  __shared__ float red[4];
  const int h = blockIdx.x, row = blockIdx.y, tid = threadIdx.x;
  const int pos = a.pos[row], slot = a.slot[row];
  const float* in = a.in + (size_t)row * a.ld;
  float *sv = ls_smem, *sk = sv + a.vp, *sq = sk + a.np, *sd = sq + a.np, *so = sd + a.np;
  const size_t hs = (size_t)a.np * a.vp, half = (size_t)a.slots * a.H * hs;
  float* st = a.state + ((size_t)slot * a.H + h) * hs;
  const float* src = st + ((pos - 1) & 1) * half;
  float* dst = st + (pos & 1) * half;
  const int c4 = a.vp >> 2, nr = 256 / c4, col = 4 * (tid % c4), r0 = tid / c4;
  constexpr int U = 8;
  // the state's first rows are on their way while the operands are formed
  float4 s0[U];
  auto fetch = [&](int n0) {
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int n = n0 + u * nr;
      s0[u] = make_float4(0.f, 0.f, 0.f, 0.f);
      if (pos > 0 && r0 < nr && n < a.np) s0[u] = *(const float4*)(src + (size_t)n * a.vp + col);
    }
  };
  fetch(r0);
  if constexpr (KEY) {
    for (int j = tid; j < a.vp; j += 256) sv[j] = j < a.dv ? in[a.v_off + h * a.dv + j] : 0.f;
    for (int n = tid; n < a.np; n += 256) {
      float d = 0.f, k = 0.f, q = 0.f;
      if (n < a.N) {
        const int c = h * a.N + n;
        float z = a.a2_b[c];
#pragma unroll 8
        for (int r = 0; r < a.rank; ++r) z = fmaf(a.a2[(size_t)c * a.rank + r], in[a.a_off + r], z);
        d = expf(-ls_softplus(-z) * a.inv_tau);
        k = in[a.k_off + c];
        q = in[a.q_off + c] * a.q_scale;
      }
      sd[n] = d;
      sk[n] = k;
      sq[n] = q;
    }
  } else {
    const float dt = lin_step_dt(a, in, h), dec = expf(-expf(a.a_log[h]) * dt);
    lin_step_conv<F32>(a, in, h, pos, slot, [&](int i, float u) {
      if (i < a.vp) {
        sv[i] = u;
      } else if (i < a.vp + a.np) {
        sk[i - a.vp] = u * dt;
        sd[i - a.vp] = dec;
      } else {
        sq[i - a.vp - a.np] = u;
      }
    });
  }
  __syncthreads();
  float4 o = make_float4(0.f, 0.f, 0.f, 0.f);
  if (r0 < nr) {
    const float4 v = *(const float4*)(sv + col);
    for (int n0 = r0; n0 < a.np; n0 += U * nr) {
      if (n0 != r0) fetch(n0);
#pragma unroll
      for (int u = 0; u < U; ++u) {
        const int n = n0 + u * nr;
        if (n >= a.np) break;
        const float d = sd[n], k = sk[n], q = sq[n];
        float4 s = s0[u];
        s.x = fmaf(d, s.x, k * v.x); s.y = fmaf(d, s.y, k * v.y); s.z = fmaf(d, s.z, k * v.z); s.w = fmaf(d, s.w, k * v.w);
        *(float4*)(dst + (size_t)n * a.vp + col) = s;
        o.x = fmaf(q, s.x, o.x); o.y = fmaf(q, s.y, o.y); o.z = fmaf(q, s.z, o.z); o.w = fmaf(q, s.w, o.w);
      }
    }
    *(float4*)(so + r0 * a.vp + col) = o;
  }
  __syncthreads();
  if constexpr (!KEY) {
    for (int j = tid; j < a.dv; j += 256) {
      float y = a.D[h] * sv[j];
      for (int r = 0; r < nr; ++r) y += so[r * a.vp + j];
      a.y[(size_t)row * a.H * a.dv + h * a.dv + j] = y;
    }
  } else {
    float ss = 0.f;
    for (int j = tid; j < a.dv; j += 256) {
      float y = 0.f;
      for (int r = 0; r < nr; ++r) y += so[r * a.vp + j];
      sv[j] = y;
      ss += y * y;
    }
    lin_step_norm<F32>(a, in, h, row, sv, ss, red);
  }
}

// ---- norm and output gate ----------------------------------------------------------------------------
// LANES threads per part of `n` numbers (64: four parts a workgroup, 256: one); PER pieces of V numbers a thread
template <bool F32, bool KEY, int LANES, int PER, int V>
__global__ void __launch_bounds__(256) lin_norm_kernel(LinScanArgs a, int parts, int n) {
  __shared__ float red[4];
  const int per = 256 / LANES, p = blockIdx.x * per + (int)threadIdx.x / LANES, lane = threadIdx.x % LANES, row = blockIdx.y;
  if (LANES == 64 && p >= parts) return;
  const int c0 = p * n;
  const float* y = a.y + (size_t)row * a.H * a.dv + c0;
  const float* z = a.in + (size_t)row * a.ld + a.z_off + c0;
  const float* nw = a.norm_w + (KEY ? 0 : c0);
  typedef float vec __attribute__((ext_vector_type(V)));
  vec v[PER], gt[PER], w[PER];
  float ss = 0.f;
#pragma unroll
  for (int i = 0; i < PER; ++i) {
    const int c = V * (lane + LANES * i);
    v[i] = gt[i] = w[i] = vec(0.f);
    if (c < n) {
      v[i] = *(const vec*)(y + c);
      gt[i] = *(const vec*)(z + c);
      w[i] = *(const vec*)(nw + c);
    }
  }
#pragma unroll
  for (int i = 0; i < PER; ++i)
#pragma unroll
    for (int e = 0; e < V; ++e) {
      gt[i][e] = ls_silu<F32>(gt[i][e]);
      if constexpr (!KEY) v[i][e] *= gt[i][e];
      ss += v[i][e] * v[i][e];
    }
  if constexpr (LANES == 64) {
#pragma unroll
    for (int d = 32; d; d >>= 1) ss += __shfl_xor(ss, d, 64);
  } else {
    ss = lin_block_sum(ss, red);
  }
  const float inv = a.out_scale / sqrtf(ss / (float)n + a.eps);
#pragma unroll
  for (int i = 0; i < PER; ++i) {
    const int c = V * (lane + LANES * i);
    if (c >= n) break;
    vec o = v[i] * inv * w[i];
    if constexpr (KEY) o *= gt[i];
    const size_t at = (size_t)row * a.ldo + c0 + c;
    if constexpr (V == 1) put1<F32>(a.out, at, o[0]);
    else if constexpr (F32) *(vec*)((float*)a.out + at) = o;
    else *(lu2*)((bf16_t*)a.out + at) = lu2{pk_bf16(o[0], o[1]), pk_bf16(o[2], o[3])};
  }
}

template <bool F32, bool KEY, int V>
static void lin_norm_v(const LinScanArgs& a, hipStream_t st) {
  const int parts = KEY ? a.H : a.norm_parts, n = a.H * a.dv / parts, m = (n + V - 1) / V;
  auto wave = [&](auto per) {
    hipLaunchKernelGGL((lin_norm_kernel<F32, KEY, 64, decltype(per)::value, V>), dim3((parts + 3) / 4, a.rows), dim3(256), 0, st, a,
                       parts, n);
  };
  auto block = [&](auto per) {
    hipLaunchKernelGGL((lin_norm_kernel<F32, KEY, 256, decltype(per)::value, V>), dim3(parts, a.rows), dim3(256), 0, st, a, parts,
                       n);
  };
  if (m <= 64) wave(std::integral_constant<int, 1>{});
  else if (m <= 128) wave(std::integral_constant<int, 2>{});
  else if (m <= 256) block(std::integral_constant<int, 1>{});
  else if (m <= 512) block(std::integral_constant<int, 2>{});
  else if (m <= 1024) block(std::integral_constant<int, 4>{});
  else if (m <= 2048) block(std::integral_constant<int, 8>{});
  else if (m <= 4096) block(std::integral_constant<int, 16>{});
  else block(std::integral_constant<int, 64>{});
}

template <bool F32, bool KEY>
static void lin_norm(const LinScanArgs& a, hipStream_t st) {
  const int n = a.H * a.dv / (KEY ? a.H : a.norm_parts);
  const bool wide = n % 4 == 0 && a.ld % 4 == 0 && a.z_off % 4 == 0 && a.ldo % 4 == 0 && ((uintptr_t)a.out & 15) == 0;
  if (wide) lin_norm_v<F32, KEY, 4>(a, st);
  else lin_norm_v<F32, KEY, 1>(a, st);
}

template <bool F32, int KIND>
static void lin_go(const LinScanArgs& a, hipStream_t st) {
  constexpr bool KEY = KIND == LIN_KEY, DELTA = KIND == LIN_DELTA;
  if (!a.seqs && DELTA) return launch_delta_step(a, st);
  if (!a.seqs) {
    const size_t lds = (size_t)(a.vp + 3 * a.np + 256 / (a.vp / 4) * a.vp) * 4;
    hipLaunchKernelGGL((lin_step_kernel<F32, KEY>), dim3(a.H, a.n), dim3(256), lds, st, a);
    if (!KEY) lin_norm<F32, KEY>(a, st);
    return;
  }
  const int nblk = 2 * a.n_chunks;
  auto walk = [&](auto nt) {
    constexpr int NT = decltype(nt)::value;
    if constexpr (KEY) {
      const size_t lds = (size_t)(3 * 16 * 16 * NT + 16 * a.rank) * 4;
      if (lds > 150 * 1024) throw std::runtime_error("linear scan: decay projection too wide");
      hipLaunchKernelGGL((lin_key_prep_kernel<F32, NT>), dim3(a.H, nblk), dim3(256), lds, st, a);
    }
    const int wg = (a.H * (a.vp / 16) + 3) / 4;
    if (a.nseg > 1)
      hipLaunchKernelGGL((lin_walk_kernel<F32, KEY, NT, true>), dim3(wg, a.n_seqs, a.nseg - 1), dim3(256), 0, st, a);
    hipLaunchKernelGGL((lin_walk_kernel<F32, KEY, NT, false>), dim3(wg, a.n_seqs, a.nseg), dim3(256), 0, st, a);
  };
  if constexpr (!KEY) {
    const dim3 grid((a.H * a.vp + 2 * a.G * a.np + LC_T - 1) / LC_T, DELTA ? a.n_chunks : nblk);
    if (a.taps <= 4) hipLaunchKernelGGL((lin_conv_kernel<F32, 4, DELTA>), grid, dim3(LC_T), 0, st, a);
    else hipLaunchKernelGGL((lin_conv_kernel<F32, 16, DELTA>), grid, dim3(LC_T), 0, st, a);
    if constexpr (DELTA) {
      launch_delta_walk(a, st);
      return lin_norm<F32, true>(a, st);
    }
    const int nscore = (nblk * a.H + 3) / 4, nkeep = (a.H * a.dv + 2 * a.G * a.N + 255) / 256;
    hipLaunchKernelGGL((lin_score_kernel<F32>), dim3(nscore + nkeep * a.n_seqs), dim3(256), 0, st, a, nscore, nkeep);
  }
  switch (a.np / 16) {
    case 2: walk(std::integral_constant<int, 2>{}); break;
    case 4: walk(std::integral_constant<int, 4>{}); break;
    case 6: walk(std::integral_constant<int, 6>{}); break;
    case 8: walk(std::integral_constant<int, 8>{}); break;
    case 12: walk(std::integral_constant<int, 12>{}); break;
    default: walk(std::integral_constant<int, 16>{}); break;
  }
  lin_norm<F32, KEY>(a, st);
}

// segments a portion of at most `blocks` blocks is walked in: as many waves as the chip holds
int lin_segments(int kind, int H, int np, int vp, int n_seqs, int blocks) {
  if (kind == LIN_DELTA) return 1;  // (a segment's transition is a whole matrix)
  const int waves = std::max(1, H * (vp / 16) * n_seqs), want = 1024 * lin_waves(kind == LIN_KEY, np / 16);
  return std::max(1, std::min({(want + waves / 2) / waves, LIN_SEGS / std::max(1, n_seqs), blocks / LIN_SEG_MIN, 8}));
}

void launch_lin_scan(const LinScanArgs& a, hipStream_t st) {
  const bool key = a.kind == LIN_KEY;
  if (a.H < 1 || a.G < 1 || a.H % a.G || (key && a.G != a.H) || a.np != lin_pad_n(a.N) || !a.np || a.vp % 16 || a.vp < a.dv ||
      a.vp > 1024)
    throw std::runtime_error("linear scan: bad sizes");
  if (!key && (a.taps < 1 || a.taps > 16)) throw std::runtime_error("linear scan: bad convolution");
  if (a.kind == LIN_HEAD && (a.norm_parts < 1 || (a.H * a.dv) % a.norm_parts || a.H * a.dv / a.norm_parts > 16384))
    throw std::runtime_error("linear scan: bad norm");
  if ((a.seqs ? a.n_seqs : a.n) < 1) return;
  if (a.kind == LIN_DELTA && a.seqs && a.nseg != 1) throw std::runtime_error("linear scan: the delta rule takes one segment");
  if (a.seqs && (a.nseg < 1 || (a.nseg > 1 && (!a.seg || !a.seg_dec || a.nseg * a.n_seqs > LIN_SEGS))))
    throw std::runtime_error("linear scan: bad segments");
  switch (a.kind) {
    case LIN_KEY: return a.f32 ? lin_go<true, LIN_KEY>(a, st) : lin_go<false, LIN_KEY>(a, st);
    case LIN_DELTA: return a.f32 ? lin_go<true, LIN_DELTA>(a, st) : lin_go<false, LIN_DELTA>(a, st);
    case LIN_HEAD: return a.f32 ? lin_go<true, LIN_HEAD>(a, st) : lin_go<false, LIN_HEAD>(a, st);
    default: throw std::runtime_error("linear scan: unknown kind");
  }
}

// ---- activation with a bias, fp32 --------------------------------------------------------------------
__global__ void __launch_bounds__(256) bias_act_f32_kernel(const float* x, int ldx, const float* bias, float* y, int ldy, int n,
                                                           int act, ActNum num) {
  const int c = blockIdx.x * 256 + threadIdx.x;
  if (c >= n) return;
  float v = x[(size_t)blockIdx.y * ldx + c] + (bias ? bias[c] : 0.f);
  if (act == ACT_RELU2) {
    v = fmaxf(v, 0.f);
    v *= v;
  } else if (act == ACT_XIELU) {
    const float m = fminf(v, 0.f);
    v = 0.5f * v + (v > 0.f ? num.pos * v * v : num.neg * (expm1f(m) - m));
  } else {
    const float u = act == ACT_GELU_TANH ? 1.5957691216057308f * fmaf(0.044715f * v * v, v, v) : v;
    v = v / (1.f + expf(-u));
  }
  y[(size_t)blockIdx.y * ldy + c] = num.scale * v;
}

void launch_bias_act_f32(const float* x, int ldx, const float* bias, float* y, int ldy, int rows, int n, int act, const ActNum& num,
                         hipStream_t st) {
  if (rows < 1 || n < 1) return;
  hipLaunchKernelGGL(bias_act_f32_kernel, dim3((n + 255) / 256, rows), dim3(256), 0, st, x, ldx, bias, y, ldy, n, act, num);
}

}  // namespace aios
