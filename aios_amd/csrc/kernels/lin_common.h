// Device helpers shared by the linear recurrences' kernels (linear_scan.hip, delta_rule.hip).
#pragma once
#include "../mixers.h"
#include "gemm_common.h"

namespace aios {

typedef unsigned int lu2 __attribute__((ext_vector_type(2)));

template <bool F32>
__device__ __forceinline__ float ls_exp(float x) { return F32 ? expf(x) : __expf(x); }
template <bool F32>
__device__ __forceinline__ float ls_silu(float z) { return z / (1.f + ls_exp<F32>(-z)); }
// log(1 + e^z)
__device__ __forceinline__ float ls_softplus(float z) { return fmaxf(z, 0.f) + log1pf(expf(-fabsf(z))); }

// two floats -> bf16 pairs (hi) and what the rounding left (lo)
__device__ __forceinline__ void split2(float a, float b, uint32_t& hi, uint32_t& lo) {
  hi = pk_bf16(a, b);
  lo = pk_bf16(a - __uint_as_float(hi << 16), b - __uint_as_float(hi & 0xffff0000u));
}
__device__ __forceinline__ void split4(gf32x4 v, lu2& hi, lu2& lo) {
  uint32_t h0, l0, h1, l1;
  split2(v[0], v[1], h0, l0);
  split2(v[2], v[3], h1, l1);
  hi = lu2{h0, h1};
  lo = lu2{l0, l1};
}
__device__ __forceinline__ gf32x4 mfma32(lu2 a0, lu2 a1, lu2 b0, lu2 b1, gf32x4 c) {
  return __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(gbf16x8, make_uint4(a0.x, a0.y, a1.x, a1.y)),
                                                 __builtin_bit_cast(gbf16x8, make_uint4(b0.x, b0.y, b1.x, b1.y)), c, 0, 0, 0);
}
// one 16-deep product in fp32: step r takes the depths 4 (lane / 16) + r
__device__ __forceinline__ gf32x4 mfma4(gf32x4 a, gf32x4 b, gf32x4 c) {
#pragma unroll
  for (int r = 0; r < 4; ++r) c = __builtin_amdgcn_mfma_f32_16x16x4f32(a[r], b[r], c, 0, 0, 0);
  return c;
}

// 16 numbers of one row of an operand
template <bool F32>
__device__ __forceinline__ void put16(void* base, size_t at, const float (&v)[16]) {
  if constexpr (F32) {
#pragma unroll
    for (int i = 0; i < 16; i += 4) *(float4*)((float*)base + at + i) = make_float4(v[i], v[i + 1], v[i + 2], v[i + 3]);
  } else {
    uint32_t u[8];
#pragma unroll
    for (int i = 0; i < 8; ++i) u[i] = pk_bf16(v[2 * i], v[2 * i + 1]);
    *(uint4*)((bf16_t*)base + at) = make_uint4(u[0], u[1], u[2], u[3]);
    *(uint4*)((bf16_t*)base + at + 8) = make_uint4(u[4], u[5], u[6], u[7]);
  }
}
template <bool F32>
__device__ __forceinline__ void put1(void* base, size_t at, float v) {
  if constexpr (F32) ((float*)base)[at] = v;
  else ((bf16_t*)base)[at] = f32_to_bf16(v);
}

// Operands of delta_rule.hip are ordered so that the eight numbers a lane takes into a 32-deep product are neighbours: token t
// of channel i in a block's and group's rows (a column's 32 tokens: four of the first block, the same four of the second, ..)
__device__ __forceinline__ size_t pair_row(int i, int t) {
  return (i >> 5) * 512 + t * 32 + ((i >> 2) & 3) * 8 + ((i >> 4) & 1) * 4 + (i & 3);
}

// a block's rows of the step
struct LinBlock {
  int row0, n, slot, pos0, seq_pos0;  // seq_pos0: the portion's first position
};
__device__ __forceinline__ LinBlock lin_block(const LinScanArgs& a, int b) {
  const ScanChunk c = a.chunks[b >> 1];
  const int t0 = (b & 1) * LIN_T;
  return LinBlock{c.row0 + t0, min(LIN_T, c.n - t0), c.slot, c.pos0 + t0, a.chunks[c.first].pos0};
}

// workgroup k of nkeep per portion: the portion's last inputs of the convolution into the ring (the convolution, which reads it,
// is a launch before this one)
__device__ __forceinline__ void lin_keep(const LinScanArgs& a, int k, int nkeep) {
  const int C = a.H * a.dv + 2 * a.G * a.N;
  const ScanSeq s = a.seqs[k / nkeep];
  const int c = (k % nkeep) * 256 + threadIdx.x;
  if (c >= C) return;
  for (int i = 0; i < min(s.n, a.taps); ++i) {
    const int t = s.n - 1 - i;
    a.ring[((size_t)s.slot * a.taps + (s.pos0 + t) % a.taps) * C + c] = a.in[(size_t)(s.row0 + t) * a.ld + a.x_off + c];
  }
}

// sum over the workgroup (red: 4 floats)
__device__ __forceinline__ float lin_block_sum(float v, float* red) {
#pragma unroll
  for (int d = 32; d; d >>= 1) v += __shfl_xor(v, d, 64);
  __syncthreads();
  if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = v;
  __syncthreads();
  float t = 0.f;
  for (int i = 0; i < ((int)blockDim.x >> 6); ++i) t += red[i];
  return t;
}

// the convolution of a token's columns for head h: put(i, value) for v's [0, vp), k's [vp, vp + np) and q's [vp + np, vp + 2 np)
template <bool F32, class Put>
__device__ __forceinline__ void lin_step_conv(const LinScanArgs& a, const float* in, int h, int pos, int slot, Put put) {
  const int C = a.H * a.dv + 2 * a.G * a.N, rep = a.H / a.G, g = h / rep, p0 = pos % a.taps;
  for (int i = threadIdx.x; i < a.vp + 2 * a.np; i += 256) {
    int raw = -1;
    if (i < a.vp) {
      if (i < a.dv) raw = h * a.dv + i;
    } else {
      const int sec = i >= a.vp + a.np, n = i - a.vp - sec * a.np;
      if (n < a.N) raw = a.H * a.dv + (sec * a.G + g) * a.N + n;
    }
    float u = 0.f;
    if (raw >= 0) {
      const float x = in[a.x_off + raw];
      u = fmaf(a.conv_w[(size_t)raw * a.taps + a.taps - 1], x, a.conv_b ? a.conv_b[raw] : 0.f);
      float* ring = a.ring + (size_t)slot * a.taps * C + raw;
#pragma unroll 4
      for (int d = 1; d < a.taps; ++d) {
        const int e = p0 - d + (p0 < d ? a.taps : 0);
        const float xd = ring[(size_t)e * C];
        u = fmaf(a.conv_w[(size_t)raw * a.taps + a.taps - 1 - d], d <= pos ? xd : 0.f, u);
      }
      u = ls_silu<F32>(u);
      // (k and q are the group's: its first head keeps them; nobody reads this position's entry in this launch)
      if (i < a.vp || h % rep == 0) ring[(size_t)p0 * C] = x;
    }
    put(i, u);
  }
}
__device__ __forceinline__ float lin_step_dt(const LinScanArgs& a, const float* in, int h) {
  return ls_softplus(in[a.dt_off + h] + a.dt_b[h]);
}

// root mean square of a head's dv numbers in y (LDS), weight, output gate -> out
template <bool F32>
__device__ __forceinline__ void lin_step_norm(const LinScanArgs& a, const float* in, int h, int row, const float* y, float ss, float* red) {
  const float inv = a.out_scale / sqrtf(lin_block_sum(ss, red) / (float)a.dv + a.eps);
  for (int j = threadIdx.x; j < a.dv; j += 256)
    put1<F32>(a.out, (size_t)row * a.ldo + h * a.dv + j, y[j] * inv * a.norm_w[j] * ls_silu<F32>(in[a.z_off + h * a.dv + j]));
}

// delta_rule.hip: LIN_DELTA's part of a portion between the convolution and the norm, and its single tokens
void launch_delta_walk(const LinScanArgs& a, hipStream_t st);
void launch_delta_step(const LinScanArgs& a, hipStream_t st);

}  // namespace aios
