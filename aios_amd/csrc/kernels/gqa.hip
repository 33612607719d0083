// Grouped-query attention of the layered decoders (mixers.h GqaArgs) over a paged cache: soft cap, sink, window or
// chunks, a gate per head.
//
//   gqa_prep   biases, norms, rotation, mixing of values, queries (the score's factor folded in) and the cache's new keys
//              and values
//   gqa_attn   rows of one sequence that read the same key / value head, 16 to a tile (the query heads of a token,
//              then further tokens): S^T = K Q^T per 32-key tile and wave, P^T goes from the accumulators into
//              O^T += V^T P^T without leaving registers (V through a wave's own slice of LDS); the four waves take the
//              tiles in turn and meet at the end.  Keys may be split over workgroups; gqa_combine sums the splits.
// Long portions take the flash kernel (attention_mha.hip) instead.  Scores, weights and sums are fp32; the weights enter
// the value product as two bf16 terms (hi + lo).
#include <algorithm>
#include <stdexcept>

#include "../mixers.h"
#include "gemm_common.h"

namespace aios {

typedef short qv4i16 __attribute__((ext_vector_type(4)));
typedef unsigned int qu32x4 __attribute__((ext_vector_type(4)));

constexpr float Q_LOG2E = 1.4426950408889634f;

// without a cap the scores come out in log2 units; with one as the exponent (log2 units) of tanh's exponential
float gqa_q_factor(float scale, float softcap) { return softcap > 0.f ? 2.f * Q_LOG2E * scale / softcap : Q_LOG2E * scale; }

bool gqa_supports(int dkp, int dvp) { return dkp > 0 && dvp > 0 && dkp <= 256 && dvp <= 256 && dkp % 32 == 0 && dvp % 32 == 0; }

__device__ __forceinline__ int gqa_low(const GqaArgs& a, int pos) {  // first visible key
  int low = a.chunk ? pos - pos % a.chunk : 0;
  if (a.window) low = max(low, pos - a.window + 1);
  return low;
}

// ---- prep ---------------------------------------------------------------------------------------
template <bool F32>
__global__ void __launch_bounds__(256) gqa_prep_kernel(GqaArgs a, float qf) {
  const int row = blockIdx.x, pos = a.pos[row], slot = a.slot[row];
  const float* in = a.in + (size_t)row * a.ld;
  const size_t blk = (size_t)a.bt[(size_t)slot * a.maxb + pos / GQA_BLOCK] * a.G * GQA_BLOCK * (a.dkp + a.dvp);
  const int key = pos % GQA_BLOCK, half = a.rot >> 1, hp = a.dkp >> 1;
  const int nq = a.H * hp, nk = nq + a.G * hp, nall = nk + a.G * (a.dvp >> 1);
  const float2* cs = a.rope + (size_t)pos * half;
  auto put = [](void* base, size_t i, float v) {
    if constexpr (F32) ((float*)base)[i] = v;
    else ((bf16_t*)base)[i] = f32_to_bf16(v);
  };
  for (int i = blockIdx.y * 256 + threadIdx.x; i < nall; i += 256 * gridDim.y) {
    if (i >= nk) {
      const int v = i - nk, g = v / (a.dvp >> 1), c = 2 * (v - g * (a.dvp >> 1));
      const size_t at = blk + (size_t)a.G * GQA_BLOCK * a.dkp + ((size_t)g * GQA_BLOCK + key) * a.dvp + c;
#pragma unroll
      for (int e = 0; e < 2; ++e) {
        float x = 0.f;
        if (c + e < a.dv) x = in[a.v_off + g * a.dv + c + e] + (a.vb ? a.vb[g * a.dv + c + e] : 0.f);
        put(a.pool, at + e, x);
      }
      continue;
    }
    const bool isq = i < nq;
    const int k = isq ? i : i - nq, h = k / hp, j = k - h * hp;
    const float* x = in + (isq ? a.q_off : a.k_off) + h * a.dk;
    const float* b = isq ? a.qb : a.kb;
    const int c0 = j < half ? j : a.rot + 2 * (j - half), c1 = j < half ? j + half : c0 + 1;
    float u = c0 < a.dk ? x[c0] + (b ? b[h * a.dk + c0] : 0.f) : 0.f;
    float v = c1 < a.dk ? x[c1] + (b ? b[h * a.dk + c1] : 0.f) : 0.f;
    if (j < half) {
      const float2 t = cs[j];
      const float p = u * t.x - v * t.y;
      v = v * t.x + u * t.y;
      u = p;
    }
    if (isq) {
      const size_t at = ((size_t)row * a.H + h) * a.dkp;
      put(a.q, at + c0, F32 ? u : u * qf);
      put(a.q, at + c1, F32 ? v : v * qf);
    } else {
      const size_t at = blk + ((size_t)h * GQA_BLOCK + key) * a.dkp;
      put(a.pool, at + c0, u);
      put(a.pool, at + c1, v);
    }
  }
}

// with norms of q, k or v, numbers per head or mixed values: workgroups y < nq take a row's queries (each sums them all for the
// norm and writes its share), y = nq its keys, the others four heads' values, a wave each
template <bool F32>
__global__ void __launch_bounds__(256) gqa_norm_prep_kernel(GqaArgs a, float qf, int nq) {
  __shared__ float red[4];
  const int row = blockIdx.x, y = blockIdx.y, tid = threadIdx.x, pos = a.pos[row], slot = a.slot[row], key = pos % GQA_BLOCK;
  const float* in = a.in + (size_t)row * a.ld;
  const size_t blk = (size_t)a.bt[(size_t)slot * a.maxb + pos / GQA_BLOCK] * a.G * GQA_BLOCK * (a.dkp + a.dvp);
  if (y > nq) {
    const int g = (y - nq - 1) * 4 + (tid >> 6), lane = tid & 63;
    if (g >= a.G) return;
    float v[4], ss = 0.f;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int c = lane + 64 * i;
      v[i] = 0.f;
      if (c < a.dv) v[i] = in[a.v_off + g * a.dv + c] + (a.vb ? a.vb[g * a.dv + c] : 0.f);
      ss = fmaf(v[i], v[i], ss);
    }
#pragma unroll
    for (int d = 32; d; d >>= 1) ss += __shfl_xor(ss, d, 64);
    const float inv = a.v_norm ? 1.f / sqrtf(ss / (float)a.dv + a.eps) : 1.f, lam = a.lambda ? *a.lambda : 0.f;
    const size_t at = blk + (size_t)a.G * GQA_BLOCK * a.dkp + ((size_t)g * GQA_BLOCK + key) * a.dvp;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int c = lane + 64 * i;
      if (c >= a.dvp) break;
      float x = v[i] * inv;
      if (a.first && c < a.dv) {
        float* f = a.first + ((size_t)row * a.G + g) * a.dv + c;
        if (a.lambda) x = (1.f - lam) * x + lam * *f;
        else *f = x;
      }
      if constexpr (F32) ((float*)a.pool)[at + c] = x;
      else ((bf16_t*)a.pool)[at + c] = f32_to_bf16(x);
    }
    return;
  }
  const bool isq = y < nq;
  const int heads = isq ? a.H : a.G, n = heads * a.dk, half = a.rot >> 1;
  const float *x = in + (isq ? a.q_off : a.k_off), *b = isq ? a.qb : a.kb, *w = isq ? a.qn : a.kn;
  const float2* cs = a.rope + (size_t)pos * half;
  const bool vec = ((a.dk | a.ld | a.q_off | a.k_off) & 3) == 0;  // (whole 16-byte pieces)
  float inv = 1.f;
  if (w) {
    float ss = 0.f;
    if (vec) {
      for (int i = 4 * tid; i < n; i += 1024) {
        gf32x4 u = *(const gf32x4*)(x + i);
        if (b) u += *(const gf32x4*)(b + i);
        ss += (u[0] * u[0] + u[1] * u[1]) + (u[2] * u[2] + u[3] * u[3]);
      }
    } else {
      for (int i = tid; i < n; i += 256) {
        const float u = x[i] + (b ? b[i] : 0.f);
        ss = fmaf(u, u, ss);
      }
    }
#pragma unroll
    for (int d = 32; d; d >>= 1) ss += __shfl_xor(ss, d, 64);
    if ((tid & 63) == 0) red[tid >> 6] = ss;
    __syncthreads();
    inv = 1.f / sqrtf(((red[0] + red[1]) + (red[2] + red[3])) / (float)n + a.eps);
  }
  auto at = [&](int i) { return (x[i] + (b ? b[i] : 0.f)) * inv * (w ? w[i] : 1.f); };
  for (int i = 4 * ((isq ? y * 256 : 0) + tid); i < heads * a.dkp; i += 1024 * (isq ? nq : 1)) {
    const int h = i / a.dkp, c = i - h * a.dkp, k = h * a.dk + c;  // (padded head sizes are whole fours)
    gf32x4 u = {0.f, 0.f, 0.f, 0.f};
    if (vec && c < a.dk) {
      u = *(const gf32x4*)(x + k);
      if (b) u += *(const gf32x4*)(b + k);
      u *= inv;
      if (w) u *= *(const gf32x4*)(w + k);
    } else {
#pragma unroll
      for (int e = 0; e < 4; ++e)
        if (c + e < a.dk) u[e] = at(k + e);
    }
    if (c < a.rot) {
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const int j = c + e;
        if (j >= a.rot) break;
        const float2 t = cs[j < half ? j : j - half];
        u[e] = j < half ? u[e] * t.x - at(k + e + half) * t.y : u[e] * t.x + at(k + e - half) * t.y;
      }
    }
    if (isq) {
      u *= (a.temp ? a.temp[h] : 1.f) * (F32 ? 1.f : qf);
      const size_t o = ((size_t)row * a.H + h) * a.dkp + c;
      if constexpr (F32) *(gf32x4*)((float*)a.q + o) = u;
      else *(uint2*)((bf16_t*)a.q + o) = make_uint2(pk_bf16(u[0], u[1]), pk_bf16(u[2], u[3]));
    } else {
      const size_t o = blk + ((size_t)h * GQA_BLOCK + key) * a.dkp + c;
      if constexpr (F32) *(gf32x4*)((float*)a.pool + o) = u;
      else *(uint2*)((bf16_t*)a.pool + o) = make_uint2(pk_bf16(u[0], u[1]), pk_bf16(u[2], u[3]));
    }
  }
}

void launch_gqa_prep(const GqaArgs& a, hipStream_t st) {
  if (a.rows < 1) return;
  if (!gqa_supports(a.dkp, a.dvp) || a.H % a.G || a.rot % 2 || a.rot > a.dk || (a.rot && !a.rope))
    throw std::runtime_error("gqa: bad sizes");
  if (a.lambda && !a.first) throw std::runtime_error("gqa: no values to mix with");
  if (a.qn || a.kn || a.temp || a.v_norm || a.first) {
    const int nq = a.rows <= 64 ? (a.H * a.dkp + 1023) / 1024 : 1;
    const dim3 grid(a.rows, nq + 1 + (a.G + 3) / 4);
    if (a.f32) hipLaunchKernelGGL((gqa_norm_prep_kernel<true>), grid, dim3(256), 0, st, a, 1.f, nq);
    else hipLaunchKernelGGL((gqa_norm_prep_kernel<false>), grid, dim3(256), 0, st, a, gqa_q_factor(a.scale, a.softcap), nq);
    return;
  }
  const int pieces = ((a.H + a.G) * (a.dkp / 2) + a.G * (a.dvp / 2) + 255) / 256;
  const dim3 grid(a.rows, a.rows <= 64 ? pieces : (pieces + 3) / 4);
  if (a.f32) hipLaunchKernelGGL((gqa_prep_kernel<true>), grid, dim3(256), 0, st, a, 1.f);
  else hipLaunchKernelGGL((gqa_prep_kernel<false>), grid, dim3(256), 0, st, a, gqa_q_factor(a.scale, a.softcap));
}

// ---- attention ------------------------------------------------------------------------------------
// o (unnormalised, four columns from d) of a row -> out; M, L: maximum (log2 units) and sum without the sink
template <bool F32>
__device__ __forceinline__ void gqa_finish(const GqaArgs& a, int row, int h, int d, float4 o, float M, float L) {
  if (a.sink) {
    const float s = a.sink[h] * Q_LOG2E;
    if (s > M) {
      const float r = __builtin_amdgcn_exp2f(M - s);
      o.x *= r; o.y *= r; o.z *= r; o.w *= r;
      L = L * r + 1.f;
    } else {
      L += __builtin_amdgcn_exp2f(s - M);
    }
  }
  float f = a.out_scale / L;
  if (a.g_off >= 0) f *= 1.f / (1.f + __expf(-a.in[(size_t)row * a.ld + a.g_off + h]));
  const size_t at = (size_t)row * a.ldo + (size_t)h * a.dvp + d;
  if constexpr (F32) *(float4*)((float*)a.out + at) = make_float4(o.x * f, o.y * f, o.z * f, o.w * f);
  else *(uint2*)((bf16_t*)a.out + at) = make_uint2(pk_bf16(o.x * f, o.y * f), pk_bf16(o.z * f, o.w * f));
}

constexpr int GQ_KT = 32;  // keys per tile: half a cache block

__device__ __forceinline__ LatentTile gqa_tile(const GqaArgs& a, int t, int rep) {
  if (a.tiles) return a.tiles[t];
  const int tpt = (rep + 15) >> 4, tok = t / tpt, i = t - tok * tpt;
  return LatentTile{tok * rep + 16 * i, min(16, rep - 16 * i)};
}

template <int DK, int DV>
__global__ void __launch_bounds__(256) __attribute__((amdgpu_waves_per_eu(DK + DV <= 256 ? 2 : 1)))
gqa_attn_kernel(GqaArgs a) {
  constexpr int KS = DK / 32, OT = DV / 16, VROW = DV + 16, PPK = DV / 8, VPL = GQ_KT * PPK / 64;
  constexpr int SLICE = GQ_KT * VROW;  // bf16 per wave
  extern __shared__ __attribute__((aligned(16))) uint8_t gq_smem[];
  __shared__ float sml[4][16][2];
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int r16 = lane & 15, q = lane >> 4, rep = a.H / a.G;
  bf16_t* sV = (bf16_t*)gq_smem + wave * SLICE;
  // tiles of a portion that read the same keys are neighbours: they go to one XCD (workgroups are dealt round-robin)
  const int per_split = a.n_tiles * a.G, total = per_split * a.nsplit, per_xcd = (total + 7) >> 3;
  const int w = (blockIdx.x & 7) * per_xcd + (blockIdx.x >> 3);
  if ((int)(blockIdx.x >> 3) >= per_xcd || w >= total) return;
  const int split = w / per_split, g = (w - split * per_split) / a.n_tiles;
  const LatentTile tl = gqa_tile(a, w - split * per_split - g * a.n_tiles, rep);
  const int nf = a.n * a.H;
  const int row0 = tl.f0 / rep, len = a.pos[(tl.f0 + tl.nv - 1) / rep] + 1;
  const int* bt = a.bt + (size_t)a.slot[row0] * a.maxb;
  const int klo = gqa_low(a, a.pos[row0]) / GQ_KT, nkt = (len + GQ_KT - 1) / GQ_KT;
  const int per = (nkt - klo + a.nsplit - 1) / a.nsplit;
  const int kt0 = klo + split * per, kt1 = min(kt0 + per, nkt);
  auto flat = [&](int r) { const int f = tl.f0 + r, t = f / rep; return t * a.H + g * rep + (f - t * rep); };
  if (kt0 >= kt1) {  // (whole workgroup, before any barrier)
    if (tid < tl.nv) *(float2*)(a.ml + ((size_t)split * nf + flat(tid)) * 2) = make_float2(-INFINITY, 0.f);
    return;
  }
  const size_t belems = (size_t)a.G * GQA_BLOCK * (a.dkp + a.dvp);
  const bf16_t* kb = (const bf16_t*)a.pool + ((size_t)g * GQA_BLOCK + r16) * a.dkp + 8 * q;
  const bf16_t* vb = (const bf16_t*)a.pool + (size_t)a.G * GQA_BLOCK * a.dkp + (size_t)g * GQA_BLOCK * a.dvp;
  struct Tile {
    qu32x4 k[2][KS], v[VPL];
  };
  int next = bt[min(kt0 + wave, kt1 - 1) >> 1];  // block of the tile that is requested next
  auto load = [&](Tile& t, int kt) {
    kt = min(kt, kt1 - 1);  // (the pipeline's tail requests are re-reads)
    const size_t base = (size_t)next * belems;
    const int key0 = (kt & 1) * GQ_KT;
    next = bt[min(kt + 4, kt1 - 1) >> 1];
#pragma unroll
    for (int b = 0; b < 2; ++b)
#pragma unroll
      for (int s = 0; s < KS; ++s) {
        t.k[b][s] = qu32x4{0, 0, 0, 0};
        if (32 * s < a.dkp) t.k[b][s] = *(const qu32x4*)(kb + base + (size_t)(key0 + 16 * b) * a.dkp + 32 * s);
      }
#pragma unroll
    for (int i = 0; i < VPL; ++i) {
      const int idx = lane + 64 * i, key = idx / PPK, c = idx % PPK;
      t.v[i] = qu32x4{0, 0, 0, 0};
      if (8 * c < a.dvp) t.v[i] = *(const qu32x4*)(vb + base + (size_t)(key0 + key) * a.dvp + 8 * c);
    }
  };
  const int fq = flat(min(r16, tl.nv - 1)), mypos = a.pos[fq / a.H], mylow = gqa_low(a, mypos);
  gbf16x8 qf[KS];
  {
    const bf16_t* qp = (const bf16_t*)a.q + (size_t)fq * a.dkp + 8 * q;
#pragma unroll
    for (int s = 0; s < KS; ++s) {
      qu32x4 u = {0, 0, 0, 0};
      if (32 * s < a.dkp) u = *(const qu32x4*)(qp + 32 * s);
      qf[s] = __builtin_bit_cast(gbf16x8, u);
    }
  }
  gf32x4 o[OT];  // columns 16 t + 4 q + j, row r16
#pragma unroll
  for (int t = 0; t < OT; ++t) o[t] = gf32x4{0.f, 0.f, 0.f, 0.f};
  float m_run = -INFINITY, l_run = 0.f;
  const float cl = a.softcap * Q_LOG2E;
  auto step = [&](int kt, const Tile& tile) {
    // a wave's slice of LDS is its own and LDS executes a wave's accesses in order; the fences keep the compiler to it
    __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
#pragma unroll
    for (int i = 0; i < VPL; ++i) {
      const int idx = lane + 64 * i;
      *(qu32x4*)(sV + (idx / PPK) * VROW + (idx % PPK) * 8) = tile.v[i];
    }
    __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
    gf32x4 s4[2] = {{0.f, 0.f, 0.f, 0.f}, {0.f, 0.f, 0.f, 0.f}};
#pragma unroll
    for (int s = 0; s < KS; ++s)
#pragma unroll
      for (int b = 0; b < 2; ++b)
        s4[b] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(gbf16x8, tile.k[b][s]), qf[s], s4[b], 0, 0, 0);
    // keys 16 b + 4 q + j of row r16
    const int key0 = kt * GQ_KT + 4 * q;
    float p[8], mx = -INFINITY;
#pragma unroll
    for (int i = 0; i < 8; ++i) {
      const int key = key0 + 16 * (i >> 2) + (i & 3);
      float v = s4[i >> 2][i & 3];
      if (a.softcap > 0.f) v = fmaf(-2.f * cl, __builtin_amdgcn_rcpf(__builtin_amdgcn_exp2f(v) + 1.f), cl);
      p[i] = key <= mypos && key >= mylow ? v : -INFINITY;
      mx = fmaxf(mx, p[i]);
    }
    mx = fmaxf(mx, __shfl_xor(mx, 16, 64));
    mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
    const float mn = fmaxf(m_run, mx), ms = mn == -INFINITY ? 0.f : mn;
    const float alpha = __builtin_amdgcn_exp2f(m_run - ms);
    float ps = 0.f;
    gbf16x8 ph, pl;
#pragma unroll
    for (int i = 0; i < 8; ++i) {
      const float e = __builtin_amdgcn_exp2f(p[i] - ms);
      ps += e;
      const __bf16 hi = (__bf16)e;
      ph[i] = hi;
      pl[i] = (__bf16)(e - (float)hi);
    }
    l_run = l_run * alpha + ps;  // (this lane's keys; the four lanes of a row are summed at the end)
    if (__any(mn != m_run)) {
#pragma unroll
      for (int t = 0; t < OT; ++t) o[t] *= alpha;
    }
    m_run = mn;
    // lane 4 i + c of a 16-lane group addresses key 4 q + i (then 16 + 4 q + i), columns 4 c .. + 3, and receives
    // column r16 of the four keys
    const bf16_t* va = sV + (4 * q + (r16 >> 2)) * VROW + 4 * (r16 & 3);
#pragma unroll
    for (int t = 0; t < OT; ++t) {
      const qv4i16 x0 = __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) qv4i16*)(va + 16 * t));
      const qv4i16 x1 =
          __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) qv4i16*)(va + 16 * t + 16 * VROW));
      const gbf16x8 vf = __builtin_bit_cast(gbf16x8, __builtin_shufflevector(x0, x1, 0, 1, 2, 3, 4, 5, 6, 7));
      o[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf, ph, o[t], 0, 0, 0);
      o[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf, pl, o[t], 0, 0, 0);
    }
  };
  if (kt0 + wave < kt1) {
    Tile A, B;
    load(A, kt0 + wave);
    for (int kt = kt0 + wave; kt < kt1; kt += 8) {
      load(B, kt + 4);
      step(kt, A);
      if (kt + 4 >= kt1) break;
      load(A, kt + 8);
      step(kt + 4, B);
    }
  }
  l_run += __shfl_xor(l_run, 16, 64);
  l_run += __shfl_xor(l_run, 32, 64);
  // the four waves' sums of a row: [row][column] fp32 over the V slices
  float* so = (float*)gq_smem;
  constexpr int OS = SLICE / 2;  // floats per wave
  static_assert(OS >= 16 * DV, "shape");
  __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
#pragma unroll
  for (int t = 0; t < OT; ++t) *(gf32x4*)(so + wave * OS + r16 * DV + 16 * t + 4 * q) = o[t];
  if (q == 0) {
    sml[wave][r16][0] = m_run;
    sml[wave][r16][1] = l_run;
  }
  __syncthreads();
  const int cols = a.dvp >> 2;
  for (int i = tid; i < tl.nv * cols; i += 256) {
    const int r = i / cols, c = 4 * (i - r * cols);
    float M = -INFINITY, L = 0.f;
#pragma unroll
    for (int v = 0; v < 4; ++v) M = fmaxf(M, sml[v][r][0]);
    const float ms = M == -INFINITY ? 0.f : M;
    float4 s = make_float4(0.f, 0.f, 0.f, 0.f);
#pragma unroll
    for (int v = 0; v < 4; ++v) {
      const float e = __builtin_amdgcn_exp2f(sml[v][r][0] - ms);
      const float4 x = *(const float4*)(so + v * OS + r * DV + c);
      L += e * sml[v][r][1];
      s.x = fmaf(e, x.x, s.x); s.y = fmaf(e, x.y, s.y); s.z = fmaf(e, x.z, s.z); s.w = fmaf(e, x.w, s.w);
    }
    const int F = flat(r);
    if (a.nsplit == 1) {
      gqa_finish<false>(a, F / a.H, F % a.H, c, s, M, L);
    } else {
      *(float4*)(a.opart + ((size_t)split * nf + F) * a.dvp + c) = s;
      if (c == 0) *(float2*)(a.ml + ((size_t)split * nf + F) * 2) = make_float2(M, L);
    }
  }
}

// one wave per (row, head): lane s holds split s's maximum and sum; lane groups of dvp / 4 take the splits in turn
__global__ void __launch_bounds__(256) gqa_combine_kernel(GqaArgs a) {
  const int lane = threadIdx.x & 63, F = blockIdx.x * 4 + (threadIdx.x >> 6), nf = a.n * a.H;
  if (F >= nf) return;
  float m = -INFINITY, l = 0.f;
  if (lane < a.nsplit) {
    const float2 v = *(const float2*)(a.ml + ((size_t)lane * nf + F) * 2);
    m = v.x;
    l = v.y;
  }
  float M = m;
#pragma unroll
  for (int d = 32; d; d >>= 1) M = fmaxf(M, __shfl_xor(M, d, 64));
  const float wt = m == -INFINITY ? 0.f : __builtin_amdgcn_exp2f(m - M);
  float L = l * wt;
#pragma unroll
  for (int d = 32; d; d >>= 1) L += __shfl_xor(L, d, 64);
  const int cols = a.dvp >> 2, groups = 64 / cols, grp = lane / cols, c = 4 * (lane - grp * cols);
  float4 o = make_float4(0.f, 0.f, 0.f, 0.f);
  for (int s0 = 0; s0 < a.nsplit; s0 += groups) {
    const int s = s0 + grp;
    const float w = __shfl(wt, s & 63, 64);
    if (s < a.nsplit && grp < groups && w != 0.f) {  // (an empty split has left no sums)
      const float4 x = *(const float4*)(a.opart + ((size_t)s * nf + F) * a.dvp + c);
      o.x = fmaf(w, x.x, o.x); o.y = fmaf(w, x.y, o.y); o.z = fmaf(w, x.z, o.z); o.w = fmaf(w, x.w, o.w);
    }
  }
  float4 t = o;
  for (int k = 1; k < groups; ++k) {
    const int src = (lane + k * cols) & 63;
    t.x += __shfl(o.x, src, 64); t.y += __shfl(o.y, src, 64); t.z += __shfl(o.z, src, 64); t.w += __shfl(o.w, src, 64);
  }
  if (lane < cols) gqa_finish<false>(a, F / a.H, F % a.H, c, t, M, L);
}

// fp32: one workgroup per (row, head), 256 keys at a time: a thread per key, then a thread per column
__global__ void __launch_bounds__(256) gqa_attn_f32_kernel(GqaArgs a) {
  __shared__ float sq[256], sp[256], red[4];
  const int F = blockIdx.x, row = F / a.H, h = F - row * a.H, g = h / (a.H / a.G), tid = threadIdx.x;
  const int pos = a.pos[row], low = gqa_low(a, pos);
  const int* bt = a.bt + (size_t)a.slot[row] * a.maxb;
  const size_t belems = (size_t)a.G * GQA_BLOCK * (a.dkp + a.dvp);
  const float* pool = (const float*)a.pool;
  if (tid < a.dkp) sq[tid] = ((const float*)a.q)[(size_t)F * a.dkp + tid];
  float m = a.sink ? a.sink[h] : -INFINITY, l = a.sink ? 1.f : 0.f, o = 0.f;
  for (int k0 = low; k0 <= pos; k0 += 256) {
    __syncthreads();
    const int key = k0 + tid;
    float s = -INFINITY;
    if (key <= pos) {
      const float* kr = pool + (size_t)bt[key / GQA_BLOCK] * belems + ((size_t)g * GQA_BLOCK + key % GQA_BLOCK) * a.dkp;
      float x = 0.f;
      for (int d = 0; d < a.dk; ++d) x = fmaf(sq[d], kr[d], x);
      s = x * a.scale;
      if (a.softcap > 0.f) s = a.softcap * tanhf(s / a.softcap);
    }
    float mx = s;
#pragma unroll
    for (int d = 32; d; d >>= 1) mx = fmaxf(mx, __shfl_xor(mx, d, 64));
    if ((tid & 63) == 0) red[tid >> 6] = mx;
    __syncthreads();
    const float mn = fmaxf(m, fmaxf(fmaxf(red[0], red[1]), fmaxf(red[2], red[3])));
    const float alpha = expf(m - mn), p = expf(s - mn);
    sp[tid] = p;
    float ps = p;
#pragma unroll
    for (int d = 32; d; d >>= 1) ps += __shfl_xor(ps, d, 64);
    __syncthreads();
    if ((tid & 63) == 0) red[tid >> 6] = ps;
    __syncthreads();
    l = l * alpha + (red[0] + red[1]) + (red[2] + red[3]);
    m = mn;
    if (tid < a.dv) {
      o *= alpha;
      const int n = min(256, pos - k0 + 1);
      for (int k = 0; k < n; ++k) {
        const int key = k0 + k;
        o = fmaf(sp[k], pool[(size_t)bt[key / GQA_BLOCK] * belems + (size_t)a.G * GQA_BLOCK * a.dkp +
                             ((size_t)g * GQA_BLOCK + key % GQA_BLOCK) * a.dvp + tid], o);
      }
    }
  }
  if (tid >= a.dvp) return;
  float f = a.out_scale / l;
  if (a.g_off >= 0) f *= 1.f / (1.f + expf(-a.in[(size_t)row * a.ld + a.g_off + h]));
  ((float*)a.out)[(size_t)row * a.ldo + (size_t)h * a.dvp + tid] = tid < a.dv ? o * f : 0.f;
}

template <int DK, int DV>
static void gqa_go(const GqaArgs& a, hipStream_t st) {
  constexpr size_t lds = (size_t)4 * GQ_KT * (DV + 16) * 2;
  static_assert(lds <= 150 * 1024, "LDS");
  const int total = a.n_tiles * a.G * a.nsplit;
  hipLaunchKernelGGL((gqa_attn_kernel<DK, DV>), dim3((total + 7) / 8 * 8), dim3(256), lds, st, a);
}
template <int DK>
static void gqa_dv(const GqaArgs& a, hipStream_t st) {
  if (a.dvp <= 64) gqa_go<DK, 64>(a, st);
  else if (a.dvp <= 128) gqa_go<DK, 128>(a, st);
  else gqa_go<DK, 256>(a, st);
}

void launch_gqa_attn(const GqaArgs& a, hipStream_t st) {
  if (a.n < 1) return;
  if (!gqa_supports(a.dkp, a.dvp) || a.H % a.G || a.ldo % 4) throw std::runtime_error("gqa: bad sizes");
  if (a.f32) {
    hipLaunchKernelGGL(gqa_attn_f32_kernel, dim3(a.n * a.H), dim3(256), 0, st, a);
    return;
  }
  if (a.n_tiles < 1 || a.nsplit < 1 || a.nsplit > 64) throw std::runtime_error("gqa: bad tiles");
  if (a.dkp <= 64) gqa_dv<64>(a, st);
  else if (a.dkp <= 128) gqa_dv<128>(a, st);
  else if (a.dkp <= 192) gqa_dv<192>(a, st);
  else gqa_dv<256>(a, st);
  if (a.nsplit > 1) hipLaunchKernelGGL(gqa_combine_kernel, dim3((a.n * a.H + 3) / 4), dim3(256), 0, st, a);
}

}  // namespace aios
