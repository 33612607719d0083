// Latent attention, absorbed form (latent.h), and the small launches of the layered decoders.
//
// A decode layer is three launches between the projection GEMVs:
//   latent_prep   one wave per row normalises the latent and writes it into the paged cache; further
//                 workgroups fold the queries into the latent space (q_a = Wuk_h^T q_h, MFMA with up to
//                 16 tokens as rows);
//   latent_attn   all heads share the cached vectors, so 16 (token, head) rows form one MFMA tile: the
//                 tile of c staged in LDS serves as keys (read row-major) and, through the
//                 transposed LDS reads, as values.  Keys are split over workgroups;
//   latent_out    sums the splits, normalises (the sink joins the denominator here), multiplies by
//                 Wuv_h and by the output gate (with several tokens the sum is a launch of its own,
//                 latent_combine, so that no workgroup repeats it).
// Scores, softmax weights, their sum and the latent norm are fp32.  The weights enter the value product
// as two bf16 terms (p = hi + lo, 16 significant bits), so that product adds no rounding of its own.
#include <algorithm>
#include <cmath>

#include "../latent.h"
#include "gemm_common.h"

namespace aios {

typedef short lv4i16 __attribute__((ext_vector_type(4)));
typedef short lv8i16 __attribute__((ext_vector_type(8)));
typedef unsigned int lu32x4 __attribute__((ext_vector_type(4)));

constexpr float LOG2E = 1.4426950408889634f;

__device__ __forceinline__ float lat_exp2(float x) { return __builtin_amdgcn_exp2f(x); }
__device__ __forceinline__ float sigmoid_f(float z) { return 1.f / (1.f + expf(-z)); }

// ---- prep: latent norm + cache write, query absorption --------------------------------------------
// (cos, sin) turns of the two pairs in v, whose first number is number i0 of the rotated part (i0 % 4 == 0)
__device__ __forceinline__ float4 rope4(float4 v, const float2* cs, int i0, int rot) {
  if (i0 < rot) {
    const float2 t = cs[i0 >> 1];
    const float x = v.x, y = v.y;
    v.x = x * t.x - y * t.y;
    v.y = y * t.x + x * t.y;
  }
  if (i0 + 2 < rot) {
    const float2 t = cs[(i0 >> 1) + 1];
    const float x = v.z, y = v.w;
    v.z = x * t.x - y * t.y;
    v.w = y * t.x + x * t.y;
  }
  return v;
}

// one wave per row; the row stays in registers between its sum of squares and the scaled store.  Columns between
// the rank and the rotated part are zero in x and in the weight, so only the mean's divisor knows the rank
template <bool F32>
__device__ __forceinline__ void latent_cache_row(const LatentAttnArgs& a, int row) {
  const int lane = threadIdx.x & 63;
  const float* x = a.qdg + (size_t)row * a.ld + a.dkv_off;
  const int pos = a.pos[row], slot = a.slot[row];
  float4 v[8], g[8];  // (rp <= 2048)
#pragma unroll
  for (int i = 0; i < 8; ++i) {
    const int c = 256 * i + 4 * lane;
    v[i] = g[i] = make_float4(0.f, 0.f, 0.f, 0.f);
    if (c < a.rp) {
      v[i] = *(const float4*)(x + c);
      g[i] = *(const float4*)(a.norm_w + c);
    }
  }
  const int blk = a.bt[(size_t)slot * a.maxb + pos / a.kvb];
  const int cend = a.rot ? a.roff : a.rp;
  float s = 0.f;
#pragma unroll
  for (int i = 0; i < 8; ++i)
    if (256 * i + 4 * lane < cend) s += v[i].x * v[i].x + v[i].y * v[i].y + v[i].z * v[i].z + v[i].w * v[i].w;
  s = wave_sum(s);
  const float inv = 1.f / sqrtf(s / (float)a.rank + a.eps);
  const size_t base = ((size_t)blk * a.kvb + pos % a.kvb) * a.rp;
#pragma unroll
  for (int i = 0; i < 8; ++i) {
    const int c = 256 * i + 4 * lane;
    if (c >= a.rp) break;
    float4 o = make_float4(v[i].x * inv * g[i].x, v[i].y * inv * g[i].y, v[i].z * inv * g[i].z, v[i].w * inv * g[i].w);
    if (c >= cend) o = rope4(v[i], a.rope + (size_t)pos * (a.rot >> 1), c - a.roff, a.rot);
    if constexpr (F32) *(float4*)((float*)a.pool + base + c) = o;
    else *(uint2*)((bf16_t*)a.pool + base + c) = make_uint2(pk_bf16(o.x, o.y), pk_bf16(o.z, o.w));
  }
}

// 8 consecutive floats -> one bf16x8 fragment; they are numbers i0 .. of the rotated part (i0 < 0: none of it)
__device__ __forceinline__ gbf16x8 frag_f32(const float* p, const float2* cs, int i0, int rot) {
  float4 x0 = *(const float4*)p, x1 = *(const float4*)(p + 4);
  if (i0 >= 0) {
    x0 = rope4(x0, cs, i0, rot);
    x1 = rope4(x1, cs, i0 + 4, rot);
  }
  const uint4 u = make_uint4(pk_bf16(x0.x, x0.y), pk_bf16(x0.z, x0.w), pk_bf16(x1.x, x1.y), pk_bf16(x1.z, x1.w));
  return __builtin_bit_cast(gbf16x8, u);
}

// grid: ceil(rows / 4) cache workgroups, then row tiles x heads x (rp / 64) absorb workgroups (4 waves of
// 16 latent columns each)
__global__ void __launch_bounds__(256) latent_prep_kernel(LatentAttnArgs a, int rows, int ncache) {
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  if ((int)blockIdx.x < ncache) {
    const int row = blockIdx.x * 4 + wave;
    if (row < rows) latent_cache_row<false>(a, row);
    return;
  }
  int b = blockIdx.x - ncache;
  const int nr = a.rp >> 6;
  const int rt = b % nr;
  b /= nr;
  const int h = b % a.H, mt = b / a.H;
  const int r16 = lane & 15, q = lane >> 4;
  const int m = min(mt * 16 + r16, a.n - 1);  // (clamped rows are computed and not stored)
  const int r = rt * 64 + wave * 16 + r16;
  const float* qp = a.qdg + (size_t)m * a.ld + h * a.dkp + 8 * q;
  const bf16_t* wp = a.wukT + ((size_t)h * a.rp + r) * a.dkp + 8 * q;
  const float2* cs = a.rot ? a.rope + (size_t)a.pos[m] * (a.rot >> 1) : nullptr;
  const int qrot = a.rot ? a.qrot : a.dkp;
  gf32x4 acc = {0.f, 0.f, 0.f, 0.f};
  for (int k0 = 0; k0 < a.dkp; k0 += 128) {  // (four K-steps' loads in flight together; steps past dkp re-read)
    gbf16x8 af[4], bf[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const int k = min(k0 + 32 * i, a.dkp - 32);
      bf[i] = __builtin_bit_cast(gbf16x8, *(const lu32x4*)(wp + k));
      af[i] = frag_f32(qp + k, cs, k + 8 * q - qrot, a.rot);
    }
#pragma unroll
    for (int i = 0; i < 4; ++i)
      if (k0 + 32 * i < a.dkp) acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(af[i], bf[i], acc, 0, 0, 0);
  }
  bf16_t* out = (bf16_t*)a.qa;
#pragma unroll
  for (int j = 0; j < 4; ++j) {
    const int t = mt * 16 + 4 * q + j;
    if (t < a.n) out[((size_t)t * a.H + h) * a.rp + r] = f32_to_bf16(acc[j]);
  }
}

// fp32: the same two roles; absorption as one wave per (token, head), lanes over the latent columns
__global__ void __launch_bounds__(256) latent_prep_f32_kernel(LatentAttnArgs a, int rows, int ncache) {
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63;
  if ((int)blockIdx.x < ncache) {
    const int row = blockIdx.x * 4 + wave;
    if (row < rows) latent_cache_row<true>(a, row);
    return;
  }
  const int f = (blockIdx.x - ncache) * 4 + wave;
  if (f >= a.n * a.H) return;
  const int t = f / a.H, h = f - t * a.H;
  const float* qp = a.qdg + (size_t)t * a.ld + h * a.dkp;
  const float2* cs = a.rot ? a.rope + (size_t)a.pos[t] * (a.rot >> 1) : nullptr;
  const int qrot = a.rot ? a.qrot : a.dkp;
  for (int r = lane; r < a.rp; r += 64) {
    const bf16_t* wp = a.wukT + ((size_t)h * a.rp + r) * a.dkp;
    float s = 0.f;
    for (int d = 0; d < a.dkp; d += 4) {
      float4 v = *(const float4*)(qp + d);
      if (d >= qrot) v = rope4(v, cs, d - qrot, a.rot);
      s = fmaf(v.x, bf16_to_f32(wp[d]), s);
      s = fmaf(v.y, bf16_to_f32(wp[d + 1]), s);
      s = fmaf(v.z, bf16_to_f32(wp[d + 2]), s);
      s = fmaf(v.w, bf16_to_f32(wp[d + 3]), s);
    }
    ((float*)a.qa)[(size_t)f * a.rp + r] = s;
  }
}

void launch_latent_prep(const LatentAttnArgs& a, int rows, hipStream_t st) {
  const int ncache = (rows + 3) / 4;
  if (a.f32) {
    hipLaunchKernelGGL(latent_prep_f32_kernel, dim3(ncache + (a.n * a.H + 3) / 4), dim3(256), 0, st, a, rows, ncache);
  } else {
    const int nab = (a.n + 15) / 16 * a.H * (a.rp / 64);
    hipLaunchKernelGGL(latent_prep_kernel, dim3(ncache + nab), dim3(256), 0, st, a, rows, ncache);
  }
}

// ---- attention ---------------------------------------------------------------------------------
constexpr int LT_KT = 32;  // keys per tile; a cache block is a whole number of tiles

__device__ __forceinline__ LatentTile latent_tile(const LatentAttnArgs& a, int t) {
  if (a.tiles) return a.tiles[t];
  const int tpt = (a.H + 15) >> 4, tok = t / tpt, i = t - tok * tpt;
  return LatentTile{tok * a.H + 16 * i, min(16, a.H - 16 * i)};
}

// NT: 16-column tiles of the latent per wave (rp = 64 NT).
//
// A wave owns a quarter of the latent's columns for everything: it loads and stages only that slice of the
// keys (no workgroup barrier between staging and use), forms the part of every score that the slice
// contributes, and later the slice of the value product.  The partial scores of the four waves meet in
// LDS -- the one barrier per tile; two buffers of them, so nobody waits for readers -- and every
// wave sums them and keeps the softmax state of all rows.  Two tiles are on their way to registers
// while one is computed.  Both products are formed transposed (keys x rows, columns x rows): a lane's
// column is then a query row throughout, and rescaling needs no exchange.
template <int NT>
struct LatentShape {
  static constexpr int RP = 64 * NT, CW = 16 * NT;  // latent columns, columns per wave
  static constexpr int LDR = CW + 16;               // padded LDS row of a wave's slice (bf16)
  static constexpr int SROW = LT_KT + 4;            // padded LDS row of partial scores (fp32)
  static constexpr int SLICE = LT_KT * LDR;         // bf16 per wave
  static constexpr int PART = 16 * SROW;       // floats per wave and buffer
  static constexpr size_t LDS = (size_t)4 * SLICE * 2 + (size_t)2 * 4 * PART * 4;
  static_assert(LDS <= 160 * 1024 && NT % 2 == 0, "shape");
};

template <int NT>
__global__ void __launch_bounds__(256) __attribute__((amdgpu_waves_per_eu(NT <= 8 ? 2 : 1)))
latent_attn_kernel(LatentAttnArgs a) {
  using SH = LatentShape<NT>;
  constexpr int RP = SH::RP, KS = NT / 2, LDR = SH::LDR, SROW = SH::SROW;
  constexpr int PPK = 2 * NT;             // 16-byte pieces of a key's slice
  constexpr int PPT = LT_KT * PPK / 64;   // per lane and tile
  extern __shared__ __attribute__((aligned(16))) uint8_t lat_smem[];
  const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int r16 = lane & 15, q = lane >> 4;
  bf16_t* sC = (bf16_t*)lat_smem + wave * SH::SLICE;
  float* sS = (float*)(lat_smem + (size_t)4 * SH::SLICE * 2);  // [2][4 waves][16 rows][SROW]
  // consecutive tiles of one split read the same keys (the head groups of a token, the tokens of a portion):
  // they go to one XCD (workgroups are dealt round-robin), whose L2 then serves all but the first
  const int total = a.n_tiles * a.nsplit, per_xcd = (total + 7) >> 3;
  const int w = (blockIdx.x & 7) * per_xcd + (blockIdx.x >> 3);
  if ((int)(blockIdx.x >> 3) >= per_xcd || w >= total) return;
  const int split = w / a.n_tiles;
  const LatentTile tl = latent_tile(a, w - split * a.n_tiles);
  const int nf = a.n * a.H;
  const int len = a.pos[(tl.f0 + tl.nv - 1) / a.H] + 1;
  const int* bt = a.bt + (size_t)a.slot[tl.f0 / a.H] * a.maxb;
  // (windowed: from the tile of the first key that the tile's first row sees)
  const int klo = a.window ? max(0, a.pos[tl.f0 / a.H] - a.window + 1) / LT_KT : 0;
  const int nkt = (len + LT_KT - 1) / LT_KT, per = (nkt - klo + a.nsplit - 1) / a.nsplit;
  const int kt0 = klo + split * per, kt1 = min(kt0 + per, nkt);
  float* mlp = a.ml + ((size_t)split * nf + tl.f0) * 2;
  if (kt0 >= kt1) {  // (whole workgroup, before any barrier)
    if (tid < tl.nv) *(float2*)(mlp + 2 * tid) = make_float2(-INFINITY, 0.f);
    return;
  }
  // pool rows of the first keys of 64 tiles, one a lane (a lookup between the tile loads would wait for them)
  int rows = 0, rows0 = kt0;
  auto look_up = [&](int kt) {
    rows0 = kt;
    const int k0 = min(kt + lane, kt1 - 1) * LT_KT;
    rows = bt[k0 / a.kvb] * a.kvb + k0 % a.kvb;
  };
  look_up(kt0);
  const uint8_t* pool = (const uint8_t*)a.pool + wave * (SH::CW * 2);
  const uint32_t voff = (uint32_t)(lane / PPK) * (RP * 2) + (uint32_t)(lane % PPK) * 16;
  lu32x4 ra[PPT], rb[PPT];
  auto load = [&](lu32x4(&r)[PPT], int kt) {
    kt = min(kt, kt1 - 1);  // (the pipeline's tail requests are re-reads)
    if (kt - rows0 >= 64) look_up(kt);
    const int row0 = __builtin_amdgcn_readlane(rows, kt - rows0);
    const uint8_t* base = pool + (size_t)row0 * (RP * 2);
    const int last = len - 1 - kt * LT_KT;
    if (64 % PPK == 0 && last >= LT_KT - 1) {
      static_for<PPT>([&](auto I) {
        constexpr int i = decltype(I)::value;
        r[i] = *(const lu32x4*)(base + (size_t)i * (64 / PPK) * (RP * 2) + voff);
      });
    } else {  // keys past the end re-read the last one: finite, weight 0
      static_for<PPT>([&](auto I) {
        constexpr int i = decltype(I)::value;
        const int idx = lane + 64 * i, key = min(idx / PPK, last), c = idx % PPK;
        r[i] = *(const lu32x4*)(base + (uint32_t)(key * RP + c * 8) * 2);
      });
    }
  };
  // the slice is the wave's own: LDS executes a wave's accesses in order, the fences keep the compiler to it
  auto stage = [&](const lu32x4(&r)[PPT]) {
    __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
    static_for<PPT>([&](auto I) {
      constexpr int i = decltype(I)::value;
      const int idx = lane + 64 * i, key = idx / PPK, c = idx % PPK;
      *(lu32x4*)(sC + key * LDR + c * 8) = r[i];
    });
    __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
  };
  load(ra, kt0);
  load(rb, kt0 + 1);
  gbf16x8 qf[KS];  // this wave's columns of the query rows
  const int f = tl.f0 + min(r16, tl.nv - 1);
  const int mypos = a.pos[f / a.H];
  const int mylow = a.window ? mypos - a.window + 1 : 0;  // first visible key
  {
    const bf16_t* qp = (const bf16_t*)a.qa + (size_t)f * RP + wave * SH::CW + 8 * q;
#pragma unroll
    for (int s = 0; s < KS; ++s) qf[s] = __builtin_bit_cast(gbf16x8, *(const lu32x4*)(qp + 32 * s));
  }
  gf32x4 o[NT];  // columns 16 t + 4 q + j of this wave's slice, row r16
#pragma unroll
  for (int t = 0; t < NT; ++t) o[t] = gf32x4{0.f, 0.f, 0.f, 0.f};
  float m_run = -INFINITY, l_run = 0.f;
  const float sc = a.scale * LOG2E;
  auto step = [&](int kt, lu32x4(&r)[PPT]) {  // r: tile kt + 1, then the request for kt + 3
    float* part = sS + ((kt - kt0) & 1) * 4 * SH::PART;
    // ---- this slice's share of the scores, keys 16 b + 4 q + j of row r16
    {
      gf32x4 s4[2] = {{0.f, 0.f, 0.f, 0.f}, {0.f, 0.f, 0.f, 0.f}};
      const bf16_t* kr = sC + r16 * LDR + 8 * q;
#pragma unroll
      for (int s = 0; s < KS; ++s)
#pragma unroll
        for (int b = 0; b < 2; ++b) {
          const gbf16x8 kf = __builtin_bit_cast(gbf16x8, *(const lu32x4*)(kr + 16 * b * LDR + 32 * s));
          s4[b] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf, qf[s], s4[b], 0, 0, 0);
        }
      float* pw = part + wave * SH::PART + r16 * SROW + 4 * q;
#pragma unroll
      for (int b = 0; b < 2; ++b) *(gf32x4*)(pw + 16 * b) = s4[b];
    }
    __syncthreads();
    // ---- the whole scores of row r16, keys 8 q + i; online softmax
    gbf16x8 ph, pl;
    {
      const float* pr = part + r16 * SROW + 8 * q;
      gf32x4 x0 = *(const gf32x4*)pr, x1 = *(const gf32x4*)(pr + 4);
#pragma unroll
      for (int v = 1; v < 4; ++v) {
        x0 += *(const gf32x4*)(pr + v * SH::PART);
        x1 += *(const gf32x4*)(pr + v * SH::PART + 4);
      }
      const int key0 = kt * LT_KT + 8 * q;
      float p[8];
      float mx = -INFINITY;
#pragma unroll
      for (int i = 0; i < 8; ++i) {
        const float v = i < 4 ? x0[i & 3] : x1[i & 3];
        p[i] = key0 + i <= mypos && key0 + i >= mylow ? v * sc : -INFINITY;
        mx = fmaxf(mx, p[i]);
      }
      mx = fmaxf(mx, __shfl_xor(mx, 16, 64));
      mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
      const float mn = fmaxf(m_run, mx);
      const float ms = mn == -INFINITY ? 0.f : mn;  // (a row with no visible key yet: weights exp2(-inf) = 0)
      const float alpha = lat_exp2(m_run - ms);
      float ps = 0.f;
#pragma unroll
      for (int i = 0; i < 8; ++i) {
        const float e = lat_exp2(p[i] - ms);
        ps += e;
        const __bf16 hi = (__bf16)e;
        ph[i] = hi;
        pl[i] = (__bf16)(e - (float)hi);
      }
      l_run = l_run * alpha + ps;  // (this lane's keys; the four lanes of a row are summed at the end)
      if (__any(mn != m_run)) {
#pragma unroll
        for (int t = 0; t < NT; ++t) o[t] *= alpha;
      }
      m_run = mn;
    }
    // ---- values: lane 4 i + p of a 16-lane group addresses key 8 q + i (then + 4), columns 4 p .. + 3, and
    // receives column r16 of the four keys
    const bf16_t* vb = sC + (8 * q + (r16 >> 2)) * LDR + 4 * (r16 & 3);
#pragma unroll
    for (int t = 0; t < NT; ++t) {
      const lv4i16 x0 = __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) lv4i16*)(vb + 16 * t));
      const lv4i16 x1 =
          __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) lv4i16*)(vb + 16 * t + 4 * LDR));
      const gbf16x8 vf = __builtin_bit_cast(gbf16x8, __builtin_shufflevector(x0, x1, 0, 1, 2, 3, 4, 5, 6, 7));
      o[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf, ph, o[t], 0, 0, 0);
      o[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf, pl, o[t], 0, 0, 0);
    }
    if (kt + 1 < kt1) {
      stage(r);
      load(r, kt + 3);
    }
  };
  stage(ra);
  load(ra, kt0 + 2);
  for (int kt = kt0; kt < kt1; kt += 2) {
    step(kt, rb);
    if (kt + 1 < kt1) step(kt + 1, ra);
  }
  l_run += __shfl_xor(l_run, 16, 64);
  l_run += __shfl_xor(l_run, 32, 64);
  if (r16 < tl.nv) {
    float* op = a.opart + ((size_t)split * nf + tl.f0 + r16) * RP + wave * SH::CW + 4 * q;
#pragma unroll
    for (int t = 0; t < NT; ++t) *(gf32x4*)(op + 16 * t) = o[t];
    if (wave == 0 && q == 0) *(float2*)(mlp + 2 * r16) = make_float2(m_run, l_run);
  }
}

// plain form (fp32 cache, or a rank beyond the matrix-core kernels): one workgroup per (token, head), keys
// round-robin over the waves, the latent columns over the lanes (NR = rp / 64 each)
template <int NR, bool F32>
__global__ void __launch_bounds__(256) latent_attn_plain_kernel(LatentAttnArgs a) {
  constexpr int RP = 64 * NR;
  __shared__ float sm[4], sl[4];
  extern __shared__ __attribute__((aligned(16))) float so[];  // [4][RP]
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int f = blockIdx.x, tok = f / a.H;
  const int len = a.pos[tok] + 1, nf = a.n * a.H;
  const int* bt = a.bt + (size_t)a.slot[tok] * a.maxb;
  float qv[NR], o[NR];
#pragma unroll
  for (int i = 0; i < NR; ++i) {
    const size_t qi = (size_t)f * RP + 64 * i + lane;
    qv[i] = F32 ? ((const float*)a.qa)[qi] : bf16_to_f32(((const bf16_t*)a.qa)[qi]);
    o[i] = 0.f;
  }
  float m = -INFINITY, l = 0.f;
  const float sc = a.scale * LOG2E;
  const int low = a.window ? max(0, len - a.window) : 0;
  for (int key = low + wave; key < len; key += 4) {
    const size_t base = ((size_t)bt[key / a.kvb] * a.kvb + key % a.kvb) * RP + lane;
    float c[NR], s = 0.f;
#pragma unroll
    for (int i = 0; i < NR; ++i) {
      c[i] = F32 ? ((const float*)a.pool)[base + 64 * i] : bf16_to_f32(((const bf16_t*)a.pool)[base + 64 * i]);
      s = fmaf(c[i], qv[i], s);
    }
    s = wave_sum(s) * sc;
    const float mn = fmaxf(m, s), alpha = exp2f(m - mn), p = exp2f(s - mn);
    l = l * alpha + p;
#pragma unroll
    for (int i = 0; i < NR; ++i) o[i] = fmaf(p, c[i], o[i] * alpha);
    m = mn;
  }
  if (lane == 0) {
    sm[wave] = m;
    sl[wave] = l;
  }
#pragma unroll
  for (int i = 0; i < NR; ++i) so[wave * RP + 64 * i + lane] = o[i];
  __syncthreads();
  const float M = fmaxf(fmaxf(sm[0], sm[1]), fmaxf(sm[2], sm[3]));  // (the token's own key is visible: finite)
  float w[4], L = 0.f;
#pragma unroll
  for (int k = 0; k < 4; ++k) {
    w[k] = exp2f(sm[k] - M);
    L += w[k] * sl[k];
  }
  for (int i = threadIdx.x; i < RP; i += 256)
    a.opart[(size_t)f * RP + i] = (so[i] * w[0] + so[RP + i] * w[1]) + (so[2 * RP + i] * w[2] + so[3 * RP + i] * w[3]);
  if (threadIdx.x == 0) *(float2*)(a.ml + 2 * (size_t)f) = make_float2(M, L);
  (void)nf;
}

bool latent_attn_mfma(int rp) { return rp <= 1024; }

template <int NT>
static void latent_attn_go(const LatentAttnArgs& a, hipStream_t st) {
  const unsigned grid = (unsigned)(((size_t)a.n_tiles * a.nsplit + 7) / 8 * 8);
  hipLaunchKernelGGL((latent_attn_kernel<NT>), dim3(grid), dim3(256), (LatentShape<NT>::LDS), st, a);
}
template <int NR, bool F32>
static void latent_plain_go(const LatentAttnArgs& a, hipStream_t st) {
  hipLaunchKernelGGL((latent_attn_plain_kernel<NR, F32>), dim3(a.n * a.H), dim3(256), (size_t)4 * 64 * NR * 4, st, a);
}
template <bool F32>
static void latent_plain(const LatentAttnArgs& a, hipStream_t st) {
  if (a.nsplit != 1) throw std::runtime_error("latent attention: the plain kernel does not split keys");
  switch (a.rp / 64) {
    case 2: return latent_plain_go<2, F32>(a, st);
    case 4: return latent_plain_go<4, F32>(a, st);
    case 6: return latent_plain_go<6, F32>(a, st);
    case 8: return latent_plain_go<8, F32>(a, st);
    case 10: return latent_plain_go<10, F32>(a, st);
    case 12: return latent_plain_go<12, F32>(a, st);
    case 16: return latent_plain_go<16, F32>(a, st);
    case 32: return latent_plain_go<32, F32>(a, st);
  }
  throw std::runtime_error("latent attention: unsupported padded rank " + std::to_string(a.rp));
}

void launch_latent_attn(const LatentAttnArgs& a, hipStream_t st) {
  if (a.n < 1) return;
  if (a.kvb % LT_KT) throw std::runtime_error("latent attention: cache block must be a whole number of key tiles");
  if (a.f32) return latent_plain<true>(a, st);
  switch (a.rp / 64) {
    case 2: return latent_attn_go<2>(a, st);
    case 4: return latent_attn_go<4>(a, st);
    case 6: return latent_attn_go<6>(a, st);
    case 8: return latent_attn_go<8>(a, st);
    case 10: return latent_attn_go<10>(a, st);
    case 12: return latent_attn_go<12>(a, st);
    case 16: return latent_attn_go<16>(a, st);
  }
  latent_plain<false>(a, st);
}

// ---- combine + Wuv + gate ------------------------------------------------------------------------
constexpr int LO_SMAX = 64;  // key splits at most

// softmax coefficients of (token t, head h): coef[s] = exp2(m_s - M) / (sum + sink) into c (lane s)
__device__ __forceinline__ float latent_coef(const LatentAttnArgs& a, int t, int h, int lane) {
  const size_t nf = (size_t)a.n * a.H, f = (size_t)t * a.H + h;
  float m = -INFINITY, l = 0.f;
  if (lane < a.nsplit) {
    const float2 v = *(const float2*)(a.ml + (lane * nf + f) * 2);
    m = v.x;
    l = v.y;
  }
  float M = wave_max(m);
  const float sk = a.sink ? a.sink[h] * LOG2E : -INFINITY;
  M = fmaxf(M, sk);
  const float e = exp2f(m - M);
  const float den = wave_sum(l * e) + exp2f(sk - M);
  return l > 0.f ? e / den : 0.f;
}

constexpr int LO_SB = 16;   // splits whose partial sums are in flight together
constexpr int LO_WB = 4;   // Wuv fragments in flight together

// the splits of every (token, head) summed and normalised: bf16 [n][H][rp] over the absorbed queries, which the
// attention is done with.  A thread owns four latent columns of a row; partial sums and their maxima of
// LO_SB splits are in flight together
__global__ void __launch_bounds__(256) latent_combine_kernel(LatentAttnArgs a) {
  const int q4 = a.rp >> 2;
  const size_t nf = (size_t)a.n * a.H, item = (size_t)blockIdx.x * 256 + threadIdx.x;
  if (item >= nf * q4) return;
  const size_t f = item / q4;
  const int c4 = 4 * (int)(item - f * q4);
  const float* p = a.opart + f * a.rp + c4;
  float M = -INFINITY, den = 0.f;
  float4 s = make_float4(0.f, 0.f, 0.f, 0.f);
  auto rescale = [&](float mx) {
    const float mn = fmaxf(M, mx), ms = mn == -INFINITY ? 0.f : mn, al = lat_exp2(M - ms);
    M = mn;
    den *= al;
    s.x *= al; s.y *= al; s.z *= al; s.w *= al;
    return ms;
  };
  for (int k0 = 0; k0 < a.nsplit; k0 += LO_SB) {
    float4 v[LO_SB];
    float2 ml[LO_SB];
#pragma unroll
    for (int k = 0; k < LO_SB; ++k) {
      // (a split without a key of this row holds what an earlier launch left there: finite, weight 0)
      const size_t sp = min(k0 + k, a.nsplit - 1);
      ml[k] = *(const float2*)(a.ml + (sp * nf + f) * 2);
      v[k] = *(const float4*)(p + sp * nf * a.rp);
    }
    float mx = -INFINITY;
#pragma unroll
    for (int k = 0; k < LO_SB; ++k) mx = fmaxf(mx, ml[k].x);
    const float ms = rescale(mx);
#pragma unroll
    for (int k = 0; k < LO_SB; ++k) {
      const float w = k0 + k < a.nsplit && ml[k].y > 0.f ? lat_exp2(ml[k].x - ms) : 0.f;
      den = fmaf(w, ml[k].y, den);
      s.x = fmaf(w, v[k].x, s.x); s.y = fmaf(w, v[k].y, s.y); s.z = fmaf(w, v[k].z, s.z); s.w = fmaf(w, v[k].w, s.w);
    }
  }
  if (a.sink) {
    const float sk = a.sink[f % a.H] * LOG2E, ms = rescale(sk);
    den += lat_exp2(sk - ms);
  }
  const float inv = 1.f / den;
  *(uint2*)((bf16_t*)a.qa + f * a.rp + c4) = make_uint2(pk_bf16(s.x * inv, s.y * inv), pk_bf16(s.z * inv, s.w * inv));
}

// FUSED: the combination in the same launch (single tokens: 256 small workgroups repeat it); else the rows
// latent_combine left in qa.  KW: waves that share a 16-column tile's K (4: 16 output columns per
// workgroup, for few rows; 1: 64)
template <int KW, bool FUSED>
__global__ void __launch_bounds__(256) latent_out_kernel(LatentAttnArgs a) {
  extern __shared__ __attribute__((aligned(16))) uint8_t lo_smem[];
  const int xrow = a.rp + 8;
  bf16_t* sX = (bf16_t*)lo_smem;                         // [16][rp + 8]
  float* sw = (float*)(lo_smem + (size_t)16 * xrow * 2); // [16][LO_SMAX]
  float* sred = sw + 16 * LO_SMAX;                       // [4][16][16] (KW == 4)
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int r16 = lane & 15, q = lane >> 4;
  const int h = blockIdx.y, t0 = blockIdx.z * 16;
  const int nt = min(16, a.n - t0);
  const int col = KW == 4 ? blockIdx.x * 16 + r16 : blockIdx.x * 64 + wave * 16 + r16;
  const bool cok = col < a.dvp;
  // this wave's first Wuv fragments, requested before the combination they do not depend on
  const bf16_t* wp = a.wuv + ((size_t)h * a.dvp + (cok ? col : 0)) * a.rp + 8 * q;
  const int ks = a.rp >> 5, s0 = KW == 4 ? wave : 0;
  constexpr int SD = KW == 4 ? 4 : 1;
  lu32x4 wf[LO_WB];
#pragma unroll
  for (int i = 0; i < LO_WB; ++i) wf[i] = *(const lu32x4*)(wp + 32 * min(s0 + SD * i, ks - 1));
  if constexpr (FUSED) {
    for (int m = wave; m < nt; m += 4) {
      const float c = latent_coef(a, t0 + m, h, lane);
      sw[m * LO_SMAX + lane] = c;  // (zero past the last split)
    }
    __syncthreads();
    const size_t nf = (size_t)a.n * a.H;
    const int q4 = a.rp >> 2;
    for (int idx = tid; idx < 16 * q4; idx += 256) {
      const int m = idx / q4, c4 = 4 * (idx - m * q4);
      float4 s = make_float4(0.f, 0.f, 0.f, 0.f);
      if (m < nt) {
        const float* p = a.opart + ((size_t)(t0 + m) * a.H + h) * a.rp + c4;
        for (int k0 = 0; k0 < a.nsplit; k0 += LO_SB) {
          // (a split without a key of this row holds what an earlier launch left there: finite, weight 0)
          float4 v[LO_SB];
  #pragma unroll
          for (int k = 0; k < LO_SB; ++k) v[k] = *(const float4*)(p + (size_t)min(k0 + k, a.nsplit - 1) * nf * a.rp);
  #pragma unroll
          for (int k = 0; k < LO_SB; ++k) {
            const float w = sw[m * LO_SMAX + k0 + k];
            s.x = fmaf(w, v[k].x, s.x); s.y = fmaf(w, v[k].y, s.y); s.z = fmaf(w, v[k].z, s.z); s.w = fmaf(w, v[k].w, s.w);
          }
        }
      }
      *(uint2*)(sX + m * xrow + c4) = make_uint2(pk_bf16(s.x, s.y), pk_bf16(s.z, s.w));
    }
    __syncthreads();
  }
  gf32x4 acc = {0.f, 0.f, 0.f, 0.f};
  const bf16_t* xp = FUSED ? sX + r16 * xrow + 8 * q
                           : (const bf16_t*)a.qa + ((size_t)min(t0 + r16, a.n - 1) * a.H + h) * a.rp + 8 * q;
  for (int sb = s0; sb < ks; sb += SD * LO_WB) {
    if (sb != s0)
#pragma unroll
      for (int i = 0; i < LO_WB; ++i) wf[i] = *(const lu32x4*)(wp + 32 * min(sb + SD * i, ks - 1));
#pragma unroll
    for (int i = 0; i < LO_WB; ++i) {
      const int s = sb + SD * i;
      if (s < ks) {
        const gbf16x8 af = __builtin_bit_cast(gbf16x8, *(const lu32x4*)(xp + 32 * s));
        acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(af, __builtin_bit_cast(gbf16x8, wf[i]), acc, 0, 0, 0);
      }
    }
  }
  if constexpr (KW == 4) {
#pragma unroll
    for (int j = 0; j < 4; ++j) sred[(wave * 16 + 4 * q + j) * 16 + r16] = acc[j];
    __syncthreads();
    if (wave != 0) return;
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      float s = 0.f;
#pragma unroll
      for (int w = 0; w < 4; ++w) s += sred[(w * 16 + 4 * q + j) * 16 + r16];
      acc[j] = s;
    }
  }
  if (!cok) return;
#pragma unroll
  for (int j = 0; j < 4; ++j) {
    const int t = t0 + 4 * q + j;
    if (t >= a.n) continue;
    float v = acc[j];
    const int c = h * a.dvp + col;
    if (a.g_off >= 0) v *= sigmoid_f(a.qdg[(size_t)t * a.ld + a.g_off + (a.head_gate ? h : c)]);
    ((bf16_t*)a.out)[(size_t)t * a.ldo + c] = f32_to_bf16(v);
  }
}

// fp32: one workgroup per (token, head); the normalised latent sum in LDS, one wave per value column
__global__ void __launch_bounds__(256) latent_out_f32_kernel(LatentAttnArgs a) {
  extern __shared__ __attribute__((aligned(16))) float lof_smem[];  // [rp]
  __shared__ float sw[LO_SMAX];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int f = blockIdx.x, t = f / a.H, h = f - t * a.H;
  if (wave == 0) {
    const float c = latent_coef(a, t, h, lane);
    if (lane < a.nsplit) sw[lane] = c;
  }
  __syncthreads();
  const size_t nf = (size_t)a.n * a.H;
  for (int i = threadIdx.x; i < a.rp; i += 256) {
    float s = 0.f;
    for (int k = 0; k < a.nsplit; ++k)
      if (sw[k] != 0.f) s = fmaf(sw[k], a.opart[(k * nf + f) * a.rp + i], s);
    lof_smem[i] = s;
  }
  __syncthreads();
  for (int d = wave; d < a.dvp; d += 4) {
    const bf16_t* wp = a.wuv + ((size_t)h * a.dvp + d) * a.rp;
    float s = 0.f;
    for (int i = lane; i < a.rp; i += 64) s = fmaf(bf16_to_f32(wp[i]), lof_smem[i], s);
    s = wave_sum(s);
    if (lane == 0) {
      const int c = h * a.dvp + d;
      if (a.g_off >= 0) s *= sigmoid_f(a.qdg[(size_t)t * a.ld + a.g_off + (a.head_gate ? h : c)]);
      ((float*)a.out)[(size_t)t * a.ldo + c] = s;
    }
  }
}

void launch_latent_out(const LatentAttnArgs& a, hipStream_t st) {
  if (a.n < 1) return;
  if (a.nsplit < 1 || a.nsplit > LO_SMAX) throw std::runtime_error("latent attention: bad key split");
  if (a.f32) {
    hipLaunchKernelGGL(latent_out_f32_kernel, dim3(a.n * a.H), dim3(256), (size_t)a.rp * 4, st, a);
    return;
  }
  const int zt = (a.n + 15) / 16;
  const size_t lds = (size_t)16 * (a.rp + 8) * 2 + (16 * LO_SMAX + 4 * 16 * 16) * 4;
  if (a.n == 1) {
    hipLaunchKernelGGL((latent_out_kernel<4, true>), dim3((a.dvp + 15) / 16, a.H, zt), dim3(256), lds, st, a);
    return;
  }
  const size_t items = (size_t)a.n * a.H * (a.rp / 4);
  hipLaunchKernelGGL(latent_combine_kernel, dim3((unsigned)((items + 255) / 256)), dim3(256), 0, st, a);
  if ((a.dvp + 63) / 64 * a.H * zt < 2 * device_cu_count())
    hipLaunchKernelGGL((latent_out_kernel<4, false>), dim3((a.dvp + 15) / 16, a.H, zt), dim3(256), lds, st, a);
  else
    hipLaunchKernelGGL((latent_out_kernel<1, false>), dim3((a.dvp + 63) / 64, a.H, zt), dim3(256), lds, st, a);
}

// ---- expanded form: gather -----------------------------------------------------------------------
__global__ void latent_gather_kernel(const bf16_t* __restrict__ pool, const int* __restrict__ bt, int kvb, int k0, int S,
                                     int rp, bf16_t* __restrict__ out) {
  const int p8 = rp >> 3;
  const size_t n = (size_t)S * p8;
  for (size_t i = (size_t)blockIdx.x * blockDim.x + threadIdx.x; i < n; i += (size_t)gridDim.x * blockDim.x) {
    const int key = (int)(i / p8), c = (int)(i - (size_t)key * p8);
    const int at = k0 + key;
    *(uint4*)(out + (size_t)key * rp + 8 * c) =
        *(const uint4*)(pool + ((size_t)bt[at / kvb] * kvb + at % kvb) * rp + 8 * c);
  }
}
void launch_latent_gather(const bf16_t* pool, const int* bt, int maxb, int kvb, int slot, int k0, int S, int rp, bf16_t* out,
                          hipStream_t st) {
  const size_t n = (size_t)S * (rp / 8);
  const int g = (int)std::min<size_t>(2048, (n + 255) / 256);
  hipLaunchKernelGGL(latent_gather_kernel, dim3(g), dim3(256), 0, st, pool, bt + (size_t)slot * maxb, kvb, k0, S, rp, out);
}

// ---- layered decoders: row gather, weight transpose, fp32 GLU ---------------------------
__global__ void gather_rows_kernel(const float* __restrict__ x, int d, const int* __restrict__ rows, float* __restrict__ y) {
  const float* s = x + (size_t)rows[blockIdx.x] * d;
  for (int k = threadIdx.x * 4; k < d; k += blockDim.x * 4) *(float4*)(y + (size_t)blockIdx.x * d + k) = *(const float4*)(s + k);
}
void launch_gather_rows(const float* x, int d, const int* rows, int n, float* y, hipStream_t st) {
  hipLaunchKernelGGL(gather_rows_kernel, dim3(n), dim3(256), 0, st, x, d, rows, y);
}

__global__ void transpose_heads_kernel(const bf16_t* __restrict__ w, int rows, int cols, bf16_t* __restrict__ out) {
  const size_t per = (size_t)rows * cols;
  const bf16_t* s = w + blockIdx.y * per;
  bf16_t* o = out + blockIdx.y * per;
  for (size_t i = (size_t)blockIdx.x * blockDim.x + threadIdx.x; i < per; i += (size_t)gridDim.x * blockDim.x) {
    const int r = (int)(i / cols), c = (int)(i - (size_t)r * cols);
    o[(size_t)c * rows + r] = s[i];
  }
}
void launch_transpose_heads(const bf16_t* w, int H, int rows, int cols, bf16_t* out, hipStream_t st) {
  const int g = (int)std::min<size_t>(256, ((size_t)rows * cols + 255) / 256);
  hipLaunchKernelGGL(transpose_heads_kernel, dim3(g, H), dim3(256), 0, st, w, rows, cols, out);
}

__global__ void glu_f32_kernel(const float* __restrict__ gu, int ldg, float* __restrict__ out, int ldo, int n, int act) {
  const float* g = gu + (size_t)blockIdx.y * ldg;
  float* o = out + (size_t)blockIdx.y * ldo;
  for (int i = blockIdx.x * blockDim.x + threadIdx.x; i < n; i += gridDim.x * blockDim.x) {
    const float2 v = *(const float2*)(g + 2 * i);
    const float z = v.x;
    const float u = act == ACT_GELU_TANH ? 1.5957691216057308f * fmaf(0.044715f * z * z, z, z) : z;
    o[i] = z / (1.f + expf(-u)) * v.y;
  }
}
void launch_glu_f32(const float* gu, int ldg, float* out, int ldo, int rows, int n, int act, hipStream_t st) {
  hipLaunchKernelGGL(glu_f32_kernel, dim3(std::min(64, (n + 255) / 256), rows), dim3(256), 0, st, gu, ldg, out, ldo, n, act);
}

}  // namespace aios
