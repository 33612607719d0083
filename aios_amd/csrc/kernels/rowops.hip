// Row operations of the layered decoders (mixers.h): one workgroup per row, the row in registers between
// its sums of squares and its stores, everything in fp32.
#include <algorithm>
#include <stdexcept>

#include "../mixers.h"
#include "gemm_common.h"

namespace aios {

__device__ __forceinline__ float4 bf4(uint2 u) {
  return make_float4(__uint_as_float(u.x << 16), __uint_as_float(u.x & 0xffff0000u), __uint_as_float(u.y << 16),
                     __uint_as_float(u.y & 0xffff0000u));
}
__device__ __forceinline__ float sq4(float4 v) { return (v.x * v.x + v.y * v.y) + (v.z * v.z + v.w * v.w); }
template <bool F32>
__device__ __forceinline__ void put4(void* out, size_t i, float4 v) {
  if constexpr (F32) *(float4*)((float*)out + i) = v;
  else *(uint2*)((bf16_t*)out + i) = make_uint2(pk_bf16(v.x, v.y), pk_bf16(v.z, v.w));
}
template <bool F32>
__device__ __forceinline__ float sig(float z) {
  return 1.f / (1.f + (F32 ? expf(-z) : __expf(-z)));
}

// sum over the workgroup: lane exchanges in registers, one LDS round over the waves (red: 16 floats a call)
__device__ __forceinline__ float row_sum(float v, float* red) {
  v += __uint_as_float(__builtin_amdgcn_update_dpp(0, __float_as_uint(v), 0xB1, 0xf, 0xf, true));   // quad_perm [1,0,3,2]
  v += __uint_as_float(__builtin_amdgcn_update_dpp(0, __float_as_uint(v), 0x4E, 0xf, 0xf, true));   // quad_perm [2,3,0,1]
  v += __uint_as_float(__builtin_amdgcn_update_dpp(0, __float_as_uint(v), 0x141, 0xf, 0xf, true));  // row_half_mirror
  v += __uint_as_float(__builtin_amdgcn_update_dpp(0, __float_as_uint(v), 0x140, 0xf, 0xf, true));  // row_mirror
  const auto a = __builtin_amdgcn_permlane16_swap(__float_as_uint(v), __float_as_uint(v), false, false);
  v = __uint_as_float(a[0]) + __uint_as_float(a[1]);
  const auto b = __builtin_amdgcn_permlane32_swap(__float_as_uint(v), __float_as_uint(v), false, false);
  v = __uint_as_float(b[0]) + __uint_as_float(b[1]);
  const int nw = blockDim.x >> 6;
  if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = v;
  __syncthreads();
  float t = 0.f;
  for (int i = 0; i < nw; ++i) t += red[i];
  return t;
}

// the next operand of row r from its residual v (NV float4 per thread at columns 4 (tid + i blockDim))
template <int NV, bool F32>
__device__ __forceinline__ void next_operand(const NextArgs& nx, int r, int dp, int d, float eps, const float4 (&v)[NV],
                                             float* red) {
  if (nx.kind == NEXT_NONE) return;
  float inv = 1.f;
  float4 w[NV];  // (requested before the sum it is needed after)
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int c = 4 * ((int)threadIdx.x + i * (int)blockDim.x);
    if (nx.kind == NEXT_NORM && c < dp) w[i] = *(const float4*)(nx.g + c);
  }
  if (nx.kind == NEXT_NORM) {
    float s = 0.f;
#pragma unroll
    for (int i = 0; i < NV; ++i) s += sq4(v[i]);
    inv = 1.f / sqrtf(row_sum(s, red) / (float)d + eps);
  }
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int c = 4 * ((int)threadIdx.x + i * (int)blockDim.x);
    if (c >= dp) break;
    float4 o = v[i];
    if (nx.kind == NEXT_NORM) {
      const float4 g = w[i];
      o = make_float4(o.x * inv * g.x, o.y * inv * g.y, o.z * inv * g.z, o.w * inv * g.w);
    }
    put4<F32>(nx.out, (size_t)r * nx.ldo + c, o);
  }
}

template <int NV, bool F32>
__global__ void embed_rows_kernel(EmbedArgs a) {
  __shared__ float red[16];
  const int r = blockIdx.x, tok = a.tokens[r], pos = a.pos[r];
  const bf16_t* e = a.table + (size_t)tok * a.dp;
  const bf16_t* p = a.pos_table ? a.pos_table + (size_t)pos * a.dp : nullptr;
  const bf16_t* b = nullptr;
  if (a.pair_table) {
    const int run = a.run ? a.run[r] : 1, slot = a.slot[r];
    long long row = a.buckets;
    if (pos > 0) {
      const int prev = run > 0 ? a.last[((pos - 1) & 1) * a.slots + slot] : a.tokens[r - 1];
      row = ((long long)prev * a.mul_prev + (long long)tok * a.mul_cur) % a.buckets;
      row = row < 0 ? row + a.buckets : row;
    }
    b = a.pair_table + (size_t)row * a.dp;
    if (run > 0) {
      __syncthreads();  // (everyone has read the slot's entry)
      if (threadIdx.x == 0) a.last[((pos + run - 1) & 1) * a.slots + slot] = a.tokens[r + run - 1];
    }
  }
  float4 v[NV];
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int c = 4 * ((int)threadIdx.x + i * (int)blockDim.x);
    v[i] = make_float4(0.f, 0.f, 0.f, 0.f);
    if (c >= a.dp) continue;
    v[i] = bf4(*(const uint2*)(e + c));
    v[i].x *= a.scale; v[i].y *= a.scale; v[i].z *= a.scale; v[i].w *= a.scale;
    if (p) {
      const float4 w = bf4(*(const uint2*)(p + c));
      v[i].x += w.x; v[i].y += w.y; v[i].z += w.z; v[i].w += w.w;
    }
    if (b) {
      const float4 w = bf4(*(const uint2*)(b + c));
      v[i].x += w.x; v[i].y += w.y; v[i].z += w.z; v[i].w += w.w;
    }
    *(float4*)(a.x + (size_t)r * a.dp + c) = v[i];
    if (a.keep) put4<F32>(a.keep, (size_t)r * a.ld_keep + c, v[i]);
    if (a.keep32) *(float4*)(a.keep32 + (size_t)r * a.dp + c) = v[i];
  }
  next_operand<NV, F32>(a.next, r, a.dp, a.d, a.eps, v, red);
}

template <int NV, bool F32>
__global__ void row_close_kernel(RowCloseArgs a) {
  __shared__ float red[2][16];
  const int r = blockIdx.x;
  float4 v[NV], x[NV], p[NV];
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int c = 4 * ((int)threadIdx.x + i * (int)blockDim.x);
    v[i] = x[i] = make_float4(0.f, 0.f, 0.f, 0.f);
    p[i] = make_float4(1.f, 1.f, 1.f, 1.f);
    if (c >= a.dp) continue;
    if (a.post) p[i] = *(const float4*)(a.post + c);
    const size_t at = (size_t)r * a.dp + c;
    if (a.y) v[i] = *(const float4*)(a.y + at);
    if (!a.replace) x[i] = *(const float4*)(a.x + at);
    if (a.y_bias) {
      const float4 b = *(const float4*)(a.y_bias + c);
      v[i].x += b.x; v[i].y += b.y; v[i].z += b.z; v[i].w += b.w;
    }
    if (a.ye) {
      for (int k0 = 0; k0 < a.top; k0 += 4) {
        float4 u[4];
        float w[4];
#pragma unroll
        for (int k = 0; k < 4; ++k) {  // (past the last expert: weight 0 of a row that is read anyway)
          const int kk = min(k0 + k, a.top - 1);
          w[k] = k0 + k < a.top ? a.wt[r * a.top + kk] : 0.f;
          const size_t src = (size_t)a.pair[r * a.top + kk] * a.dp + c;
          if constexpr (F32) u[k] = *(const float4*)((const float*)a.ye + src);
          else u[k] = bf4(*(const uint2*)((const bf16_t*)a.ye + src));
        }
#pragma unroll
        for (int k = 0; k < 4; ++k) {
          v[i].x = fmaf(w[k], u[k].x, v[i].x); v[i].y = fmaf(w[k], u[k].y, v[i].y);
          v[i].z = fmaf(w[k], u[k].z, v[i].z); v[i].w = fmaf(w[k], u[k].w, v[i].w);
        }
      }
    }
    if (a.gate) {
      float4 g = *(const float4*)(a.gate + (size_t)r * a.ldg + c);
      if (a.gate_bias) {
        const float4 b = *(const float4*)(a.gate_bias + c);
        g.x += b.x; g.y += b.y; g.z += b.z; g.w += b.w;
      }
      v[i].x *= sig<F32>(g.x); v[i].y *= sig<F32>(g.y); v[i].z *= sig<F32>(g.z); v[i].w *= sig<F32>(g.w);
    }
    if (a.replace && a.add) {
      const float4 b = *(const float4*)(a.add + c);
      v[i].x += b.x; v[i].y += b.y; v[i].z += b.z; v[i].w += b.w;
    }
  }
  float inv = 1.f;
  if (a.post) {
    float s = 0.f;
#pragma unroll
    for (int i = 0; i < NV; ++i) s += sq4(v[i]);
    inv = 1.f / sqrtf(row_sum(s, red[0]) / (float)a.d + a.eps);
  }
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int c = 4 * ((int)threadIdx.x + i * (int)blockDim.x);
    if (c >= a.dp) continue;
    const float4 g = p[i];
    v[i].x = x[i].x + v[i].x * inv * g.x; v[i].y = x[i].y + v[i].y * inv * g.y;
    v[i].z = x[i].z + v[i].z * inv * g.z; v[i].w = x[i].w + v[i].w * inv * g.w;
    if (a.extra) {
      const float4 b = *(const float4*)(a.extra + (size_t)r * a.dp + c);
      v[i].x += b.x; v[i].y += b.y; v[i].z += b.z; v[i].w += b.w;
    }
    *(float4*)(a.x + (size_t)r * a.dp + c) = v[i];
  }
  next_operand<NV, F32>(a.next, r, a.dp, a.d, a.eps, v, red[1]);
}

template <bool F32, typename A, typename K1, typename K2, typename K4>
static void row_go(const A& a, int dp, int rows, hipStream_t st, K1 k1, K2 k2, K4 k4) {
  if (dp % 64 || dp > 16384) throw std::runtime_error("row operation: width must be padded to 64 and at most 16384");
  if (rows < 1) return;
  const int q = dp / 4, t = std::min(1024, (q + 63) / 64 * 64), nv = (q + t - 1) / t;
  if (nv <= 1) hipLaunchKernelGGL(k1, dim3(rows), dim3(t), 0, st, a);
  else if (nv <= 2) hipLaunchKernelGGL(k2, dim3(rows), dim3(t), 0, st, a);
  else hipLaunchKernelGGL(k4, dim3(rows), dim3(t), 0, st, a);
}

void launch_embed_rows(const EmbedArgs& a, int rows, hipStream_t st) {
  if (a.pair_table && (a.buckets < 1 || !a.last)) throw std::runtime_error("embedding: bad pair table");
  if (a.f32) row_go<true>(a, a.dp, rows, st, embed_rows_kernel<1, true>, embed_rows_kernel<2, true>, embed_rows_kernel<4, true>);
  else row_go<false>(a, a.dp, rows, st, embed_rows_kernel<1, false>, embed_rows_kernel<2, false>, embed_rows_kernel<4, false>);
}

void launch_row_close(const RowCloseArgs& a, int rows, hipStream_t st) {
  if (a.ye && a.top < 1) throw std::runtime_error("row_close: expert rows without experts");
  if (a.f32) row_go<true>(a, a.dp, rows, st, row_close_kernel<1, true>, row_close_kernel<2, true>, row_close_kernel<4, true>);
  else row_go<false>(a, a.dp, rows, st, row_close_kernel<1, false>, row_close_kernel<2, false>, row_close_kernel<4, false>);
}

}  // namespace aios
