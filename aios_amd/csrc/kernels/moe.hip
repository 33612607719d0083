// Mixture of experts of the layered decoders (mixers.h).
//
//   few tokens (<= MOE_FEW)   two launches.  Every (token, expert) pair is its own matrix-vector product; the
//                             workgroups of the first repeat their token's routing (a wave, a few hundred
//                             cycles) instead of waiting for a launch that does it; the second sums a token's
//                             experts, and the shared one, into one row.
//   more                      routing and a counting sort of the pairs by expert, then two grouped products
//                             over tiles of one expert's rows: 16-row tiles streamed by waves while
//                             experts have few rows, 128 x 128 tiles through LDS beyond.
// Router scores, their softmax and the weighted sums are fp32.  A row's result does not depend on its place in
// a tile, so the order inside an expert is free.
#include <algorithm>
#include <stdexcept>

#include "../mixers.h"
#include "../latent.h"
#include "gemm_common.h"

namespace aios {

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
__device__ __forceinline__ void moe_route(const MoeArgs& a, int t, int& e, float& w) {
  if (a.experts <= 64) moe_route_token<1>(a, t, e, w);
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

// workgroup w of a grouped product with nb column blocks -> (tile, column block): an expert's tiles run
// together over each of its weight columns
__device__ __forceinline__ bool moe_place(const MoeArgs& a, int w, int nb, int4& tile, int& cb) {
  const int nt = *a.n_tiles, t = w / nb;
  if (t >= nt) return false;
  const int4 x = a.tiles[t];
  const int first = x.w & 0xffff, per = x.w >> 16, local = w - first * nb;
  cb = local / per;
  tile = a.tiles[first + local - cb * per];
  return true;
}

// ---- few tokens -------------------------------------------------------------------------------------
__device__ __forceinline__ gbf16x8 ldfrag(const bf16_t* p) { return __builtin_bit_cast(gbf16x8, *(const gu32x4*)p); }

constexpr int MF_B = 8, MF_D = 4;  // 64-column items (two MFMA steps) in flight per wave: up, down

// gate / up of every (token, expert) pair: 16 interleaved columns per workgroup, the width over its 4 waves
__global__ void __launch_bounds__(256) moe_few_up_kernel(MoeArgs a) {
  __shared__ float red[4][16];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, r16 = lane & 15, q = lane >> 4;
  const int t = blockIdx.y / a.top, k = blockIdx.y - t * a.top;
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
  const bf16_t* hp = (const bf16_t*)a.h + (size_t)t * a.ldh + 8 * q;
  gf32x4 acc = {0.f, 0.f, 0.f, 0.f};
  for (int i0 = wave; i0 < items; i0 += 4 * MF_B) {
    gbf16x8 wf[2 * MF_B], hf[2 * MF_B];
#pragma unroll
    for (int i = 0; i < MF_B; ++i) {
      const int c = 64 * min(i0 + 4 * i, items - 1);
      wf[2 * i] = ldfrag(wp + c);
      wf[2 * i + 1] = ldfrag(wp + c + 32);
      hf[2 * i] = ldfrag(hp + c);
      hf[2 * i + 1] = ldfrag(hp + c + 32);
    }
#pragma unroll
    for (int i = 0; i < MF_B; ++i)
      if (i0 + 4 * i < items) {
        acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wf[2 * i], hf[2 * i], acc, 0, 0, 0);
        acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wf[2 * i + 1], hf[2 * i + 1], acc, 0, 0, 0);
      }
  }
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

// down of a token's experts and the shared one, weighted and summed: 16 columns per workgroup, the (expert,
// 64-column) items over its 16 waves
__global__ void __launch_bounds__(1024) moe_few_down_kernel(MoeArgs a) {
  __shared__ float red[16][16];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, r16 = lane & 15, q = lane >> 4;
  const int t = blockIdx.y, row = blockIdx.x * 16 + r16;
  const int per = a.ff >> 6, routed = a.top * per, items = routed + (a.sh_dn ? a.sh_ff >> 6 : 0);
  int my_e = 0;
  float my_w = 0.f;
  if (lane < a.top) {
    my_e = a.sel[t * a.top + lane];
    my_w = a.wt[t * a.top + lane];
  }
  gf32x4 acc = {0.f, 0.f, 0.f, 0.f};
  for (int i0 = wave; i0 < items; i0 += 16 * MF_D) {
    gbf16x8 wf[2 * MF_D], hf[2 * MF_D];
    float wt[MF_D];
#pragma unroll
    for (int i = 0; i < MF_D; ++i) {
      const int it = __builtin_amdgcn_readfirstlane(min(i0 + 16 * i, items - 1));
      const bf16_t *wp, *hp;
      if (it < routed) {
        const int k = it / per, c = 64 * (it - k * per);
        const int e = __builtin_amdgcn_readlane(my_e, k);
        wt[i] = __uint_as_float(__builtin_amdgcn_readlane(__float_as_uint(my_w), k));
        wp = a.wdn + ((size_t)e * a.dp + row) * a.ff + c;
        hp = (const bf16_t*)a.act_out + ((size_t)t * a.top + k) * a.ff + c;
      } else {
        const int c = 64 * (it - routed);
        wt[i] = 1.f;
        wp = a.sh_dn + (size_t)row * a.sh_ff + c;
        hp = a.sh_act + (size_t)t * a.ld_sh + c;
      }
      wf[2 * i] = ldfrag(wp + 8 * q);
      wf[2 * i + 1] = ldfrag(wp + 8 * q + 32);
      hf[2 * i] = ldfrag(hp + 8 * q);
      hf[2 * i + 1] = ldfrag(hp + 8 * q + 32);
    }
#pragma unroll
    for (int i = 0; i < MF_D; ++i)
      if (i0 + 16 * i < items) {
        gf32x4 p = {0.f, 0.f, 0.f, 0.f};
        p = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wf[2 * i], hf[2 * i], p, 0, 0, 0);
        p = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wf[2 * i + 1], hf[2 * i + 1], p, 0, 0, 0);
#pragma unroll
        for (int j = 0; j < 4; ++j) acc[j] = fmaf(wt[i], p[j], acc[j]);
      }
  }
  if (r16 == 0) *(gf32x4*)&red[wave][4 * q] = acc;
  __syncthreads();
  if (threadIdx.x < 16) {
    float s = 0.f;
#pragma unroll
    for (int v = 0; v < 16; ++v) s += red[v][threadIdx.x];
    a.y[(size_t)t * a.dp + blockIdx.x * 16 + threadIdx.x] = s;
  }
}

static void moe_check(const MoeArgs& a) {
  if (a.experts < 1 || a.experts > MOE_MAX_EXPERTS || a.top < 1 || a.top > std::min(a.experts, MOE_MAX_TOP))
    throw std::runtime_error("moe: bad number of experts");
  if (a.dp % 64 || a.ff % 64 || a.ldh % 8 || (a.sh_dn && (a.sh_ff % 64 || a.ld_sh % 8)))
    throw std::runtime_error("moe: sizes must be padded to 64");
}

void launch_moe_few(const MoeArgs& a, hipStream_t st) {
  moe_check(a);
  if (a.f32 || a.n > MOE_FEW) throw std::runtime_error("moe: not a few-token call");
  if (a.n < 1) return;
  hipLaunchKernelGGL(moe_few_up_kernel, dim3(2 * a.ff / 16, a.n * a.top), dim3(256), 0, st, a);
  hipLaunchKernelGGL(moe_few_down_kernel, dim3(a.dp / 16, a.n), dim3(1024), 0, st, a);
}

// ---- grouped, 16-row tiles ------------------------------------------------------------------------------
// UP: rows gathered from h by token, GLU, act_out[row][ff]; else act_out -> ye.  KW: waves that share a
// 16-column block's K (4: 16 columns per workgroup; 1: 64)
constexpr int MG_B = 4;  // 64-column items in flight per wave

template <bool UP, int KW>
__global__ void __launch_bounds__(256) moe_tile16_kernel(MoeArgs a) {
  __shared__ float red[KW == 4 ? 4 : 1][16][17];
  constexpr int NB = KW == 4 ? 16 : 64;
  const int N = UP ? 2 * a.ff : a.dp, K = UP ? a.dp : a.ff;
  int4 tile;
  int cb;
  if (!moe_place(a, blockIdx.x, N / NB, tile, cb)) return;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, r16 = lane & 15, q = lane >> 4;
  const int col = cb * NB + (KW == 4 ? 0 : wave * 16);
  const int m = tile.y + min(r16, tile.z - 1);  // (rows past the tile repeat its last and are not stored)
  const bf16_t* hp = UP ? (const bf16_t*)a.h + (size_t)a.token[m] * a.ldh : (const bf16_t*)a.act_out + (size_t)m * a.ff;
  const bf16_t* wp = (UP ? a.wgu : a.wdn) + ((size_t)tile.x * N + col + r16) * K + 8 * q;
  hp += 8 * q;
  const int items = K >> 6;
  gf32x4 acc = {0.f, 0.f, 0.f, 0.f};
  for (int i0 = KW == 4 ? wave : 0; i0 < items; i0 += KW * MG_B) {
    gbf16x8 wf[2 * MG_B], hf[2 * MG_B];
#pragma unroll
    for (int i = 0; i < MG_B; ++i) {
      const int c = 64 * min(i0 + KW * i, items - 1);
      wf[2 * i] = ldfrag(wp + c);
      wf[2 * i + 1] = ldfrag(wp + c + 32);
      hf[2 * i] = ldfrag(hp + c);
      hf[2 * i + 1] = ldfrag(hp + c + 32);
    }
#pragma unroll
    for (int i = 0; i < MG_B; ++i)
      if (i0 + KW * i < items) {
        acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wf[2 * i], hf[2 * i], acc, 0, 0, 0);
        acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(wf[2 * i + 1], hf[2 * i + 1], acc, 0, 0, 0);
      }
  }
  // row r16 of the tile, columns 4 q + j
  if constexpr (KW == 4) {
#pragma unroll
    for (int j = 0; j < 4; ++j) red[wave][r16][4 * q + j] = acc[j];
    __syncthreads();
    if (wave != 0) return;
#pragma unroll
    for (int j = 0; j < 4; ++j)
      acc[j] = (red[0][r16][4 * q + j] + red[1][r16][4 * q + j]) + (red[2][r16][4 * q + j] + red[3][r16][4 * q + j]);
  }
  if (r16 >= tile.z) return;
  const size_t row = tile.y + r16;
  if constexpr (UP)
    *(uint32_t*)((bf16_t*)a.act_out + row * a.ff + (col + 4 * q) / 2) =
        pk_bf16(glu_act(acc[0], a.act) * acc[1], glu_act(acc[2], a.act) * acc[3]);
  else
    *(uint2*)((bf16_t*)a.ye + row * a.dp + col + 4 * q) = make_uint2(pk_bf16(acc[0], acc[1]), pk_bf16(acc[2], acc[3]));
}

// ---- grouped, 128 x 128 tiles -----------------------------------------------------------------------------
// Four waves of 64 x 64 (2 x 2 MFMA 32 x 32), the weights as the row operand so that a lane holds one token
// and four consecutive columns.  64-wide K steps in two LDS buffers, the next one's loads in registers.
constexpr int MB_T = 128, MB_K = 64, MB_LD = MB_K + 8;

template <bool UP>
__global__ void __launch_bounds__(256) __attribute__((amdgpu_waves_per_eu(2))) moe_tile128_kernel(MoeArgs a) {
  __shared__ __attribute__((aligned(16))) bf16_t sm[2][2][MB_T * MB_LD];
  const int N = UP ? 2 * a.ff : a.dp, K = UP ? a.dp : a.ff, nb = (N + MB_T - 1) / MB_T;
  // neighbours in work order on one XCD (workgroups are dealt round-robin over the eight)
  const int per_xcd = gridDim.x >> 3;
  int4 tile;
  int cb;
  if (!moe_place(a, (blockIdx.x & 7) * per_xcd + (blockIdx.x >> 3), nb, tile, cb)) return;
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, l32 = lane & 31, half = lane >> 5;
  const int n0 = cb * MB_T;
  const bf16_t *hp[4], *wp[4];
  const bf16_t* w0 = (UP ? a.wgu : a.wdn) + (size_t)tile.x * N * K;
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int r = (tid >> 3) + 32 * i, m = tile.y + min(r, tile.z - 1);
    hp[i] = (UP ? (const bf16_t*)a.h + (size_t)a.token[m] * a.ldh : (const bf16_t*)a.act_out + (size_t)m * a.ff) + 8 * (tid & 7);
    wp[i] = w0 + (size_t)min(n0 + r, N - 1) * K + 8 * (tid & 7);
  }
  gu32x4 rh[4], rw[4];
  auto load = [&](int k) {
    static_for<4>([&](auto I) {
      constexpr int i = decltype(I)::value;
      rh[i] = *(const gu32x4*)(hp[i] + k);
      rw[i] = *(const gu32x4*)(wp[i] + k);
    });
  };
  auto stage = [&](int b) {
    static_for<4>([&](auto I) {
      constexpr int i = decltype(I)::value;
      const int at = ((tid >> 3) + 32 * i) * MB_LD + 8 * (tid & 7);
      *(gu32x4*)(&sm[b][0][at]) = rh[i];
      *(gu32x4*)(&sm[b][1][at]) = rw[i];
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
  load(0);
  stage(0);
  __syncthreads();
  const int nk = K / MB_K;
  for (int s = 0; s < nk; ++s) {
    const int b = s & 1;
    if (s + 1 < nk) load((s + 1) * MB_K);
#pragma unroll
    for (int k = 0; k < MB_K; k += 16) {
      gbf16x8 hf[2], wf[2];
#pragma unroll
      for (int i = 0; i < 2; ++i) {
        hf[i] = ldfrag(&sm[b][0][(wm + 32 * i + l32) * MB_LD + k + 8 * half]);
        wf[i] = ldfrag(&sm[b][1][(wn + 32 * i + l32) * MB_LD + k + 8 * half]);
      }
#pragma unroll
      for (int i = 0; i < 2; ++i)
#pragma unroll
        for (int j = 0; j < 2; ++j) acc[i][j] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(wf[i], hf[j], acc[i][j], 0, 0, 0);
    }
    if (s + 1 < nk) stage(b ^ 1);
    __syncthreads();
  }
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
        const float v0 = acc[i][j][e], v1 = acc[i][j][e + 1], v2 = acc[i][j][e + 2], v3 = acc[i][j][e + 3];
        if constexpr (UP)
          *(uint32_t*)((bf16_t*)a.act_out + row * a.ff + c / 2) = pk_bf16(glu_act(v0, a.act) * v1, glu_act(v2, a.act) * v3);
        else
          *(uint2*)((bf16_t*)a.ye + row * a.dp + c) = make_uint2(pk_bf16(v0, v1), pk_bf16(v2, v3));
      }
  }
}

// average rows per expert from which the 128-row tiles pay
static int moe_big_rows() {
  static const int v = [] {
    const char* e = std::getenv("AIOS_MOE_BIG_ROWS");
    return e ? std::atoi(e) : 24;
  }();
  return v;
}
int moe_tile_rows(int n, int top, int experts) { return (double)n * top / experts >= moe_big_rows() ? MB_T : 16; }
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
  auto t16 = [&](auto up, int N) {
    constexpr bool UP = decltype(up)::value;
    if (tiles * (N / 64) >= 2 * device_cu_count())
      hipLaunchKernelGGL((moe_tile16_kernel<UP, 1>), dim3(tiles * (N / 64)), dim3(256), 0, st, a);
    else
      hipLaunchKernelGGL((moe_tile16_kernel<UP, 4>), dim3(tiles * (N / 16)), dim3(256), 0, st, a);
  };
  auto t128 = [&](auto up, int N) {
    constexpr bool UP = decltype(up)::value;
    const int grid = (tiles * ((N + MB_T - 1) / MB_T) + 7) / 8 * 8;
    hipLaunchKernelGGL((moe_tile128_kernel<UP>), dim3(grid), dim3(256), 0, st, a);
  };
  if (bm == 16) {
    t16(std::true_type{}, 2 * a.ff);
    t16(std::false_type{}, a.dp);
  } else {
    t128(std::true_type{}, 2 * a.ff);
    t128(std::false_type{}, a.dp);
  }
}

}  // namespace aios
