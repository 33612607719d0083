// Mixture of experts of the layered decoders (mixers.h).
//
//   few tokens (<= MOE_FEW)   two launches.  Every (token, expert) pair is its own matrix-vector product; the
//                             workgroups of the first repeat their token's routing (a wave, a few hundred
//                             cycles) instead of waiting for a launch that does it; the second sums a token's
//                             experts, and the shared one, into one row.
//   more                      routing and a counting sort of the pairs by expert, then two grouped products
//                             over tiles of one expert's rows: 32 rows with the weights streamed by waves
//                             while experts have few, 128 x 128 through LDS beyond.
// Router scores, their softmax and the weighted sums are fp32.  A row's result does not depend on its place in
// a tile, so the order inside an expert is free.
#include <algorithm>
#include <stdexcept>

#include "../mixers.h"
#include "../latent.h"
#include "gemm_common.h"

namespace aios {

__device__ __forceinline__ float lane_value(float v, int lane) {
  return __uint_as_float(__builtin_amdgcn_readlane(__float_as_uint(v), lane));
}

// ---- routing: one wave per token ------------------------------------------------------------------
// lane l holds experts l, l + 64, ..; NE >= experts / 64.  Lane k < top leaves with the k-th choice and its weight
template <int NE>
__device__ __forceinline__ void moe_route_token(const MoeArgs& a, int t, int& my_e, float& my_w) {
  const int lane = threadIdx.x & 63;
  float z[NE], ch[NE];
  float mx = -INFINITY;
#pragma unroll
  for (int i = 0; i < NE; ++i) {
    const int e = lane + 64 * i;
    z[i] = e < a.experts ? a.logits[(size_t)t * a.ldl + e] : -INFINITY;
    mx = fmaxf(mx, z[i]);
  }
  mx = wave_max(mx);
  float s = 0.f;
#pragma unroll
  for (int i = 0; i < NE; ++i) {
    z[i] = expf(z[i] - mx);
    s += z[i];
  }
  const float inv = 1.f / wave_sum(s);
#pragma unroll
  for (int i = 0; i < NE; ++i) {
    const int e = lane + 64 * i;
    z[i] *= inv;
    ch[i] = e < a.experts ? z[i] + (a.corr ? a.corr[e] : 0.f) : -INFINITY;
  }
  my_e = 0;
  my_w = 0.f;
  for (int k = 0; k < a.top; ++k) {
    float best = ch[0], bw = z[0];
    int bi = lane;
#pragma unroll
    for (int i = 1; i < NE; ++i)
      if (ch[i] > best) {
        best = ch[i];
        bw = z[i];
        bi = lane + 64 * i;
      }
    // the largest choice over the lanes; of equals the lowest expert
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) {
      const float ob = __shfl_xor(best, o, 64), ow = __shfl_xor(bw, o, 64);
      const int oi = __shfl_xor(bi, o, 64);
      if (ob > best || (ob == best && oi < bi)) {
        best = ob;
        bw = ow;
        bi = oi;
      }
    }
    if (lane == k) {
      my_e = bi;
      my_w = bw * a.scale;
    }
#pragma unroll
    for (int i = 0; i < NE; ++i)
      if (lane + 64 * i == bi) ch[i] = -INFINITY;
  }
}
// up to 64 experts, one a lane: an expert's place is the number of choices above its own, counted from scalar
// copies of them (no chain of lane exchanges)
__device__ __forceinline__ void moe_route_rank(const MoeArgs& a, int t, int& my_e, float& my_w) {
  const int lane = threadIdx.x & 63;
  const bool on = lane < a.experts;
  const float z = on ? a.logits[(size_t)t * a.ldl + lane] : -INFINITY;
  const float corr = on && a.corr ? a.corr[lane] : 0.f;
  float mx = -INFINITY;
  for (int e = 0; e < a.experts; ++e) mx = fmaxf(mx, lane_value(z, e));
  const float p = expf(z - mx);
  float sum = 0.f;
  for (int e = 0; e < a.experts; ++e) sum += lane_value(p, e);
  const float s = p / sum, ch = on ? s + corr : -INFINITY;
  int place = on ? 0 : 64;
  for (int e = 0; e < a.experts; ++e) {
    const float c = lane_value(ch, e);
    place += c > ch || (c == ch && e < lane);
  }
  my_e = 0;
  my_w = 0.f;
  for (int k = 0; k < a.top; ++k) {
    const int e = __ffsll(__ballot(place == k)) - 1;
    const float w = lane_value(s, e) * a.scale;
    if (lane == k) {
      my_e = e;
      my_w = w;
    }
  }
}
__device__ __forceinline__ void moe_route(const MoeArgs& a, int t, int& e, float& w) {
  if (a.experts <= 64) moe_route_rank(a, t, e, w);
  else if (a.experts <= 256) moe_route_token<4>(a, t, e, w);
  else moe_route_token<MOE_MAX_EXPERTS / 64>(a, t, e, w);
}

__global__ void __launch_bounds__(256) moe_route_kernel(MoeArgs a) {
  const int t = blockIdx.x * 4 + (threadIdx.x >> 6), lane = threadIdx.x & 63;
  if (t >= a.n) return;
  int e;
  float w;
  moe_route(a, t, e, w);
  if (lane < a.top) {
    a.sel[t * a.top + lane] = e;
    a.wt[t * a.top + lane] = w;
  }
}

// counting sort of the pairs by expert and the tile list; one workgroup.  ROUTE: the routing too (few rows)
template <bool ROUTE>
__global__ void __launch_bounds__(1024) moe_group_kernel(MoeArgs a, int bm) {
  __shared__ int cnt[MOE_MAX_EXPERTS], cur[MOE_MAX_EXPERTS];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  for (int e = tid; e < a.experts; e += 1024) cnt[e] = 0;
  if constexpr (ROUTE) {
    for (int t = wave; t < a.n; t += 16) {
      int e;
      float w;
      moe_route(a, t, e, w);
      if (lane < a.top) {
        a.sel[t * a.top + lane] = e;
        a.wt[t * a.top + lane] = w;
      }
    }
  }
  __syncthreads();  // (also orders this workgroup's own sel stores before its loads)
  const int P = a.n * a.top;
  for (int i = tid; i < P; i += 1024) atomicAdd(&cnt[a.sel[i]], 1);
  __syncthreads();
  if (wave == 0) {
    // lane l scans experts [l per, (l + 1) per)
    const int per = (a.experts + 63) / 64, e0 = min(lane * per, a.experts), e1 = min(e0 + per, a.experts);
    int rows = 0, tiles = 0;
    for (int e = e0; e < e1; ++e) {
      rows += cnt[e];
      tiles += (cnt[e] + bm - 1) / bm;
    }
    int ro = rows, to = tiles;
#pragma unroll
    for (int o = 1; o < 64; o <<= 1) {
      const int r = __shfl_up(ro, o, 64), t = __shfl_up(to, o, 64);
      if (lane >= o) {
        ro += r;
        to += t;
      }
    }
    if (lane == 63) *a.n_tiles = to;
    ro -= rows;
    to -= tiles;
    for (int e = e0; e < e1; ++e) {
      const int c = cnt[e], nt = (c + bm - 1) / bm;
      cur[e] = ro;
      for (int i = 0; i < nt; ++i) a.tiles[to + i] = make_int4(e, ro + i * bm, min(bm, c - i * bm), to | (nt << 16));
      ro += c;
      to += nt;
    }
  }
  __syncthreads();
  for (int i = tid; i < P; i += 1024) {
    const int at = atomicAdd(&cur[a.sel[i]], 1);
    a.pair[i] = at;
    a.token[at] = i / a.top;
  }
}

// workgroup of a grouped product with nb column blocks -> (tile, column block): an expert's tiles run together over
// each of its weight columns, and neighbours in that order on one XCD (workgroups are dealt round-robin over the
// eight; the grid covers the most tiles there can be, the shares are of those there are)
__device__ __forceinline__ bool moe_place(const MoeArgs& a, int nb, int4& tile, int& cb) {
  const int total = *a.n_tiles * nb, per_xcd = (total + 7) >> 3;
  const int w = (blockIdx.x & 7) * per_xcd + (blockIdx.x >> 3), t = w / nb;
  if ((int)(blockIdx.x >> 3) >= per_xcd || w >= total) return false;
  const int4 x = a.tiles[t];
  const int first = x.w & 0xffff, per = x.w >> 16, local = w - first * nb;
  cb = local / per;
  tile = a.tiles[first + local - cb * per];
  return true;
}

// ---- few tokens -------------------------------------------------------------------------------------
__device__ __forceinline__ gbf16x8 ldfrag(const bf16_t* p) { return __builtin_bit_cast(gbf16x8, *(const gu32x4*)p); }

constexpr int MF_B = 8;  // 64-column items (two MFMA steps) in flight per wave

// n bf16 numbers (a multiple of 8) into LDS
__device__ __forceinline__ void moe_stage(bf16_t* dst, const bf16_t* src, int n) {
  for (int i = 8 * threadIdx.x; i < n; i += 8 * blockDim.x) *(gu32x4*)(dst + i) = *(const gu32x4*)(src + i);
}

// gate / up of every (token, expert) pair: 16 interleaved columns per workgroup, the width over its 4 waves
__global__ void __launch_bounds__(256) moe_few_up_kernel(MoeArgs a) {
  extern __shared__ __attribute__((aligned(16))) bf16_t mf_smem[];  // the token's input [dp]
  __shared__ float red[4][16];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, r16 = lane & 15, q = lane >> 4;
  const int t = blockIdx.y / a.top, k = blockIdx.y - t * a.top;
  moe_stage(mf_smem, (const bf16_t*)a.h + (size_t)t * a.ldh, a.dp);
  int e;
  float w;
  moe_route(a, t, e, w);
  if (blockIdx.x == 0 && wave == 0 && lane == k) {
    a.sel[blockIdx.y] = e;
    a.wt[blockIdx.y] = w;
  }
  e = __builtin_amdgcn_readlane(e, k);
  const int items = a.dp >> 6;
  const bf16_t* wp = a.wgu + ((size_t)e * 2 * a.ff + blockIdx.x * 16 + r16) * a.dp + 8 * q;
  const bf16_t* hp = mf_smem + 8 * q;
  gf32x4 acc = {0.f, 0.f, 0.f, 0.f};
  for (int i0 = wave; i0 < items; i0 += 4 * MF_B) {
    gbf16x8 wf[2 * MF_B];
#pragma unroll
    for (int i = 0; i < MF_B; ++i) {
      const int c = 64 * min(i0 + 4 * i, items - 1);
      wf[2 * i] = ldfrag(wp + c);
      wf[2 * i + 1] = ldfrag(wp + c + 32);
    }
    __builtin_amdgcn_sched_barrier(0);
    if (i0 == wave) __syncthreads();  // (every wave has at least one item: the input is staged)
#pragma unroll
    for (int i = 0; i < MF_B; ++i)
      if (i0 + 4 * i < items) {
        const int c = 64 * (i0 + 4 * i);
        acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wf[2 * i], ldfrag(hp + c), acc, 0, 0, 0);
        acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wf[2 * i + 1], ldfrag(hp + c + 32), acc, 0, 0, 0);
      }
  }
  if (wave >= items) __syncthreads();
  // every lane of a quarter holds the same token: columns 4 q + j
  if (r16 == 0) *(gf32x4*)&red[wave][4 * q] = acc;
  __syncthreads();
  if (threadIdx.x < 8) {
    float v[2];
#pragma unroll
    for (int j = 0; j < 2; ++j) {
      const int c = 2 * threadIdx.x + j;
      v[j] = (red[0][c] + red[1][c]) + (red[2][c] + red[3][c]);
    }
    ((bf16_t*)a.act_out)[(size_t)blockIdx.y * a.ff + blockIdx.x * 8 + threadIdx.x] = f32_to_bf16(glu_act(v[0], a.act) * v[1]);
  }
}

// down of a token's experts and the shared one, weighted and summed: 8 columns per workgroup, two waves each.  A
// wave takes every other item of its column: 512 numbers of one expert's row, 8 a lane
constexpr int MD_B = 8;  // items in flight per wave

__device__ __forceinline__ float moe_dot8(gu32x4 w, gu32x4 x) {
  float d = 0.f;
#pragma unroll
  for (int j = 0; j < 4; ++j) {
    const uint32_t a = w[j], b = x[j];
    d = __builtin_amdgcn_fdot2_f32_bf16(__builtin_bit_cast(gbf16x2, a), __builtin_bit_cast(gbf16x2, b), d, false);
  }
  return d;
}

__global__ void __launch_bounds__(1024) moe_few_down_kernel(MoeArgs a) {
  extern __shared__ __attribute__((aligned(16))) bf16_t mf_smem[];  // activations [top][ff] | shared [sh_ff]
  __shared__ float red[16];
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int t = blockIdx.y, row = blockIdx.x * 8 + (wave >> 1);
  const int per = (a.ff + 511) >> 9, routed = a.top * per, items = routed + (a.sh_dn ? (a.sh_ff + 511) >> 9 : 0);
  int my_e = 0;
  float my_w = 0.f;
  if (lane < a.top) {
    my_e = a.sel[t * a.top + lane];
    my_w = a.wt[t * a.top + lane];
  }
  moe_stage(mf_smem, (const bf16_t*)a.act_out + (size_t)t * a.top * a.ff, a.top * a.ff);
  if (a.sh_dn) moe_stage(mf_smem + a.top * a.ff, a.sh_act + (size_t)t * a.ld_sh, a.sh_ff);
  float acc = 0.f;
  for (int i0 = wave & 1; i0 < items; i0 += 2 * MD_B) {
    gu32x4 wv[MD_B];
    float wt[MD_B];
    int at[MD_B];  // this lane's place in the staged activations
#pragma unroll
    for (int i = 0; i < MD_B; ++i) {
      const int it = i0 + 2 * i, in = min(it, items - 1);
      const bool sh = in >= routed;
      const int k = sh ? a.top : in / per, c = 512 * (in - k * per) + 8 * lane, n = sh ? a.sh_ff : a.ff;
      const int cc = min(c, n - 8);  // (past the end, as past the last item: weight 0)
      wt[i] = it < items && c < n ? (sh ? 1.f : lane_value(my_w, sh ? 0 : k)) : 0.f;
      const int e = __builtin_amdgcn_readlane(my_e, sh ? 0 : k);
      const bf16_t* base = sh ? a.sh_dn + (size_t)row * a.sh_ff : a.wdn + ((size_t)e * a.dp + row) * a.ff;
      wv[i] = *(const gu32x4*)(base + cc);
      at[i] = k * a.ff + cc;
    }
    __builtin_amdgcn_sched_barrier(0);
    if (i0 == (wave & 1)) __syncthreads();
#pragma unroll
    for (int i = 0; i < MD_B; ++i) acc = fmaf(wt[i], moe_dot8(wv[i], *(const gu32x4*)(mf_smem + at[i])), acc);
  }
  if ((wave & 1) >= items) __syncthreads();
  acc = wave_sum(acc);
  if (lane == 0) red[wave] = acc;
  __syncthreads();
  if (tid < 8) a.y[(size_t)t * a.dp + blockIdx.x * 8 + tid] = red[2 * tid] + red[2 * tid + 1];
}

static size_t moe_few_lds(const MoeArgs& a) {
  return (size_t)2 * std::max(a.dp, a.top * a.ff + (a.sh_dn ? a.sh_ff : 0));
}
bool moe_few_fits(const MoeArgs& a) { return !a.f32 && a.n <= MOE_FEW && moe_few_lds(a) <= 128 * 1024; }

static void moe_check(const MoeArgs& a) {
  if (a.experts < 1 || a.experts > MOE_MAX_EXPERTS || a.top < 1 || a.top > std::min(a.experts, MOE_MAX_TOP))
    throw std::runtime_error("moe: bad number of experts");
  if (a.dp % 64 || a.ff % 64 || a.ldh % 8 || (a.sh_dn && (a.sh_ff % 64 || a.ld_sh % 8)))
    throw std::runtime_error("moe: sizes must be padded to 64");
}

void launch_moe_few(const MoeArgs& a, hipStream_t st) {
  moe_check(a);
  if (!moe_few_fits(a)) throw std::runtime_error("moe: not a few-token call");
  if (a.n < 1) return;
  hipLaunchKernelGGL(moe_few_up_kernel, dim3(2 * a.ff / 16, a.n * a.top), dim3(256), (size_t)2 * a.dp, st, a);
  hipLaunchKernelGGL(moe_few_down_kernel, dim3(a.dp / 8, a.n), dim3(1024), moe_few_lds(a), st, a);
}

// ---- grouped products -----------------------------------------------------------------------------------
// UP: rows gathered from h by token, GLU, act_out[row][ff]; else act_out -> ye
template <bool UP>
__device__ __forceinline__ const bf16_t* moe_row(const MoeArgs& a, int r) {
  return UP ? (const bf16_t*)a.h + (size_t)a.token[r] * a.ldh : (const bf16_t*)a.act_out + (size_t)r * a.ff;
}
// columns col .. col + 3 of row `row`
template <bool UP>
__device__ __forceinline__ void moe_store(const MoeArgs& a, size_t row, int col, gf32x4 v) {
  if constexpr (UP)
    *(uint32_t*)((bf16_t*)a.act_out + row * a.ff + col / 2) = pk_bf16(glu_act(v[0], a.act) * v[1], glu_act(v[2], a.act) * v[3]);
  else
    *(uint2*)((bf16_t*)a.ye + row * a.dp + col) = make_uint2(pk_bf16(v[0], v[1]), pk_bf16(v[2], v[3]));
}

// 32-row tiles, for experts with few rows: the weights are what this reads.  They go straight to registers, one
// 256-column slice ahead, and every fragment of them serves both row fragments; the rows go through LDS (two
// buffers, one barrier a slice).  64 columns per workgroup, 16 a wave.
constexpr int MS_K = 256, MS_LD = MS_K + 16, MS_T = 32;

template <bool UP>
__global__ void __launch_bounds__(256) __attribute__((amdgpu_waves_per_eu(2))) moe_tile32_kernel(MoeArgs a) {
  constexpr int MT = MS_T / 16, RP = MS_T * MS_K / 8 / 256;  // row fragments; 16-byte row pieces per thread and slice
  __shared__ __attribute__((aligned(16))) bf16_t sm[2][MS_T * MS_LD];
  const int N = UP ? 2 * a.ff : a.dp, K = UP ? a.dp : a.ff;
  int4 tile;
  int cb;
  if (!moe_place(a, N / 64, tile, cb)) return;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, r16 = lane & 15, q = lane >> 4;
  const int col = cb * 64 + wave * 16;
  const bf16_t* wp = (UP ? a.wgu : a.wdn) + ((size_t)tile.x * N + col + r16) * K + 8 * q;
  const int pr = tid >> 5, pc = 8 * (tid & 31);  // this thread's first row (then every 8th) and column in a slice
  const bf16_t* hp[RP];
  static_for<RP>([&](auto I) {
    constexpr int i = decltype(I)::value;
    hp[i] = moe_row<UP>(a, tile.y + min(pr + 8 * i, tile.z - 1));
  });
  gu32x4 rh[RP];
  auto load_rows = [&](int k0) {
    const int c = min(k0 + pc, K - 8);  // (K is a multiple of 64: columns past it are not multiplied)
    static_for<RP>([&](auto I) {
      constexpr int i = decltype(I)::value;
      rh[i] = *(const gu32x4*)(hp[i] + c);
    });
  };
  auto stage = [&](int b) {
    static_for<RP>([&](auto I) {
      constexpr int i = decltype(I)::value;
      *(gu32x4*)(&sm[b][(pr + 8 * i) * MS_LD + pc]) = rh[i];
    });
  };
  gbf16x8 wa[8], wb[8];
  auto load_w = [&](gbf16x8(&w)[8], int k0) {
    static_for<8>([&](auto I) {
      constexpr int i = decltype(I)::value;
      w[i] = ldfrag(wp + min(k0 + 32 * i, K - 32));
    });
  };
  gf32x4 acc[MT];
#pragma unroll
  for (int m = 0; m < MT; ++m) acc[m] = gf32x4{0.f, 0.f, 0.f, 0.f};
  const int slices = (K + MS_K - 1) / MS_K;
  load_w(wa, 0);
  load_rows(0);
  stage(0);
  __syncthreads();
  auto step = [&](int s, gbf16x8(&w)[8], gbf16x8(&next)[8]) {
    if (s + 1 < slices) {
      load_w(next, (s + 1) * MS_K);
      load_rows((s + 1) * MS_K);
    }
    __builtin_amdgcn_sched_barrier(0);
    const bf16_t* x = &sm[s & 1][r16 * MS_LD + 8 * q];
    static_for<8>([&](auto I) {
      constexpr int i = decltype(I)::value;
      if (s * MS_K + 32 * i < K) {
#pragma unroll
        for (int m = 0; m < MT; ++m)
          acc[m] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(w[i], ldfrag(x + 16 * m * MS_LD + 32 * i), acc[m], 0, 0, 0);
      }
    });
    if (s + 1 < slices) stage((s + 1) & 1);
    __syncthreads();
  };
  for (int s = 0; s < slices; s += 2) {
    step(s, wa, wb);
    if (s + 1 < slices) step(s + 1, wb, wa);
  }
#pragma unroll
  for (int m = 0; m < MT; ++m)
    if (16 * m + r16 < tile.z) moe_store<UP>(a, tile.y + 16 * m + r16, col + 4 * q, acc[m]);
}

// 128 x 128 tiles: four waves of 64 x 64 (2 x 2 MFMA 32 x 32), the weights as the row operand so that a lane holds one token
// and four consecutive columns.  64-wide K steps in two LDS buffers, the loads of the three steps after the
// current one in registers.
constexpr int MB_T = 128, MB_K = 64, MB_LD = MB_K + 8;

template <bool UP>
__global__ void __launch_bounds__(256) __attribute__((amdgpu_waves_per_eu(2))) moe_tile128_kernel(MoeArgs a) {
  __shared__ __attribute__((aligned(16))) bf16_t sm[2][2][MB_T * MB_LD];
  const int N = UP ? 2 * a.ff : a.dp, K = UP ? a.dp : a.ff, nb = (N + MB_T - 1) / MB_T;
  int4 tile;
  int cb;
  if (!moe_place(a, nb, tile, cb)) return;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, l32 = lane & 31, half = lane >> 5;
  const int n0 = cb * MB_T;
  const bf16_t *hp[4], *wp[4];
  const bf16_t* w0 = (UP ? a.wgu : a.wdn) + (size_t)tile.x * N * K;
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int r = (tid >> 3) + 32 * i, m = tile.y + min(r, tile.z - 1);
    hp[i] = moe_row<UP>(a, m) + 8 * (tid & 7);
    wp[i] = w0 + (size_t)min(n0 + r, N - 1) * K + 8 * (tid & 7);
  }
  struct Regs {
    gu32x4 h[4], w[4];
  } rg[3];
  const int nk = K / MB_K;
  auto load = [&](Regs& r, int s) {
    const int k = min(s, nk - 1) * MB_K;  // (the pipeline's tail requests are re-reads)
    static_for<4>([&](auto I) {
      constexpr int i = decltype(I)::value;
      r.h[i] = *(const gu32x4*)(hp[i] + k);
      r.w[i] = *(const gu32x4*)(wp[i] + k);
    });
  };
  auto stage = [&](const Regs& r, int b) {
    static_for<4>([&](auto I) {
      constexpr int i = decltype(I)::value;
      const int at = ((tid >> 3) + 32 * i) * MB_LD + 8 * (tid & 7);
      *(gu32x4*)(&sm[b][0][at]) = r.h[i];
      *(gu32x4*)(&sm[b][1][at]) = r.w[i];
    });
  };
  const int wm = (wave >> 1) * 64, wn = (wave & 1) * 64;
  gf32x16 acc[2][2];  // [columns][rows]
#pragma unroll
  for (int i = 0; i < 2; ++i)
#pragma unroll
    for (int j = 0; j < 2; ++j)
#pragma unroll
      for (int e = 0; e < 16; ++e) acc[i][j][e] = 0.f;
  load(rg[0], 0);
  load(rg[1], 1);
  load(rg[2], 2);
  stage(rg[0], 0);
  __syncthreads();
  // (six steps a turn: both the buffers and the register sets are then fixed names, with nothing to copy or wait for
  // between steps)
  auto step = [&](auto I, int s0) {
    constexpr int i = decltype(I)::value, b = i & 1;
    load(rg[i % 3], s0 + i + 3);
    if (wm < tile.z) {  // (else none of this wave's rows exist)
#pragma unroll
      for (int k = 0; k < MB_K; k += 16) {
        gbf16x8 hf[2], wf[2];
#pragma unroll
        for (int j = 0; j < 2; ++j) {
          hf[j] = ldfrag(&sm[b][0][(wm + 32 * j + l32) * MB_LD + k + 8 * half]);
          wf[j] = ldfrag(&sm[b][1][(wn + 32 * j + l32) * MB_LD + k + 8 * half]);
        }
#pragma unroll
        for (int c = 0; c < 2; ++c)
#pragma unroll
          for (int j = 0; j < 2; ++j) acc[c][j] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(wf[c], hf[j], acc[c][j], 0, 0, 0);
      }
    }
    stage(rg[(i + 1) % 3], b ^ 1);  // (past the last step: never read)
    __syncthreads();
  };
  int s0 = 0;
  for (; s0 + 6 <= nk; s0 += 6) static_for<6>([&](auto I) { step(I, s0); });
  static_for<5>([&](auto I) {
    if (s0 + decltype(I)::value < nk) step(I, s0);
  });
#pragma unroll
  for (int j = 0; j < 2; ++j) {
    const int r = wm + 32 * j + l32;
    if (r >= tile.z) continue;
    const size_t row = tile.y + r;
#pragma unroll
    for (int i = 0; i < 2; ++i)
#pragma unroll
      for (int e = 0; e < 16; e += 4) {
        const int c = n0 + wn + 32 * i + 8 * (e >> 2) + 4 * half;
        if (c >= N) continue;
        moe_store<UP>(a, row, c, gf32x4{acc[i][j][e], acc[i][j][e + 1], acc[i][j][e + 2], acc[i][j][e + 3]});
      }
  }
}

// rows per tile by the average rows per expert (AIOS_MOE_TILE pins 32 or 128)
int moe_tile_rows(int n, int top, int experts) {
  static const int pin = [] {
    const char* e = std::getenv("AIOS_MOE_TILE");
    const int v = e ? std::atoi(e) : 0;
    return v == MS_T || v == MB_T ? v : 0;
  }();
  if (pin) return pin;
  return (double)n * top / experts <= 14 ? MS_T : MB_T;
}
int moe_max_tiles(int n, int top, int experts) {
  const int bm = moe_tile_rows(n, top, experts), p = n * top;
  return std::min(p, experts) + p / bm;
}

void launch_moe_grouped(const MoeArgs& a, hipStream_t st) {
  moe_check(a);
  if (a.n < 1) return;
  const int bm = a.f32 ? 64 : moe_tile_rows(a.n, a.top, a.experts);
  const int tiles = a.f32 ? std::min(a.n * a.top, a.experts) + a.n * a.top / 64 : moe_max_tiles(a.n, a.top, a.experts);
  if (tiles > a.max_tiles || tiles > 0xffff) throw std::runtime_error("moe: tile list too short");
  if (a.n <= 64) {
    hipLaunchKernelGGL(moe_group_kernel<true>, dim3(1), dim3(1024), 0, st, a, bm);
  } else {
    hipLaunchKernelGGL(moe_route_kernel, dim3((a.n + 3) / 4), dim3(256), 0, st, a);
    hipLaunchKernelGGL(moe_group_kernel<false>, dim3(1), dim3(1024), 0, st, a, bm);
  }
  if (a.f32) {
    launch_gemm_f32_grouped((const float*)a.h, a.ldh, a.token, a.wgu, a.tiles, a.n_tiles, tiles, 2 * a.ff, a.dp, a.gu32, st);
    launch_glu_f32(a.gu32, 2 * a.ff, (float*)a.act_out, a.ff, a.n * a.top, a.ff, a.act, st);
    launch_gemm_f32_grouped((const float*)a.act_out, a.ff, nullptr, a.wdn, a.tiles, a.n_tiles, tiles, a.dp, a.ff, (float*)a.ye, st);
    return;
  }
  const int nu = 2 * a.ff, nd = a.dp;
  auto grid = [&](int blocks) { return dim3((tiles * blocks + 7) / 8 * 8); };
  if (bm == MS_T) {
    hipLaunchKernelGGL((moe_tile32_kernel<true>), grid(nu / 64), dim3(256), 0, st, a);
    hipLaunchKernelGGL((moe_tile32_kernel<false>), grid(nd / 64), dim3(256), 0, st, a);
  } else {
    hipLaunchKernelGGL((moe_tile128_kernel<true>), grid((nu + MB_T - 1) / MB_T), dim3(256), 0, st, a);
    hipLaunchKernelGGL((moe_tile128_kernel<false>), grid((nd + MB_T - 1) / MB_T), dim3(256), 0, st, a);
  }
}

}  // namespace aios
