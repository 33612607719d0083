// minGRU recurrence of the layered decoders (mixers.h): a thread owns one channel and walks the tokens of
// one chunk, all of whose numbers it has requested before the first step.  A portion longer than a chunk takes two launches: every chunk's
// transition (S_out = a S_in + b) first, then every chunk again from the state those give it.
#include <stdexcept>

#include "../mixers.h"
#include "gemm_common.h"

namespace aios {

constexpr int MG_T = 128;  // channels per workgroup
constexpr int MG_F = 16;   // chunk transitions in flight

template <bool F32>
__device__ __forceinline__ float mg_sig(float z) {
  return 1.f / (1.f + (F32 ? expf(-z) : __expf(-z)));
}
template <bool F32>
__device__ __forceinline__ float mg_cand(float u) {
  return u >= 0.f ? u + 0.5f : mg_sig<F32>(u);
}

__device__ __forceinline__ ScanChunk mg_chunk(const MinGruArgs& a, int i) {
  if (a.chunks) return a.chunks[i];
  return ScanChunk{i, 1, a.slot[i], a.pos[i], i, 1};
}

// SCAN: the chunk's transition only.  U: tokens of a chunk at most
template <bool F32, bool SCAN, int U>
__global__ void __launch_bounds__(MG_T) mingru_kernel(MinGruArgs a) {
  const int c = blockIdx.x * MG_T + threadIdx.x;
  if (c >= a.w) return;
  const int y = blockIdx.y;
  const ScanChunk ch = mg_chunk(a, y);
  const size_t w = a.w;
  const float zb = a.zb[c], ub = a.ub[c];
  const float* in = a.in + (size_t)ch.row0 * a.ld + c;
  if (SCAN && ch.last && ch.first != y) return;  // (nobody needs its transition)
  float z[U], u[U], g[U];
#pragma unroll
  for (int i = 0; i < U; ++i) {
    const float* p = in + (size_t)min(i, ch.n - 1) * a.ld;
    z[i] = p[a.z_off];
    u[i] = p[a.u_off];
    if constexpr (!SCAN) g[i] = p[a.g_off];
  }
  __builtin_amdgcn_sched_barrier(0);
  float S = 0.f, A = 1.f;
  if (ch.first == y) {
    const float s0 = ch.pos0 > 0 ? a.state[(((ch.pos0 - 1) & 1) * (size_t)a.slots + ch.slot) * w + c] : 0.f;
    if constexpr (SCAN) {
      a.agg[((size_t)y * 3 + 2) * w + c] = s0;  // (the second launch may overwrite the slot's state)
      if (ch.last) return;
    } else {
      S = a.split ? a.agg[((size_t)y * 3 + 2) * w + c] : s0;
    }
  } else if constexpr (!SCAN) {
    S = a.agg[((size_t)ch.first * 3 + 2) * w + c];
    for (int j0 = ch.first; j0 < y; j0 += MG_F) {
      float fa[MG_F], fb[MG_F];
#pragma unroll
      for (int i = 0; i < MG_F; ++i) {
        const int j = min(j0 + i, y - 1);
        fa[i] = a.agg[((size_t)j * 3) * w + c];
        fb[i] = a.agg[((size_t)j * 3 + 1) * w + c];
      }
#pragma unroll
      for (int i = 0; i < MG_F; ++i)
        if (j0 + i < y) S = fmaf(fa[i], S, fb[i]);
    }
  }
#pragma unroll
  for (int i = 0; i < U; ++i) {
    if (i >= ch.n) break;
    const float f = mg_sig<F32>(z[i] + zb), cand = mg_cand<F32>(u[i] + ub);
    S = fmaf(f, cand - S, S);
    if constexpr (SCAN) {
      A *= 1.f - f;
    } else {
      const float o = S * g[i] * mg_sig<F32>(g[i]);
      const size_t at = (size_t)(ch.row0 + i) * a.ldo + c;
      if constexpr (F32) ((float*)a.out)[at] = o;
      else ((bf16_t*)a.out)[at] = f32_to_bf16(o);
    }
  }
  if constexpr (SCAN) {
    a.agg[((size_t)y * 3) * w + c] = A;
    a.agg[((size_t)y * 3 + 1) * w + c] = S;
  } else if (ch.last) {
    a.state[(((ch.pos0 + ch.n - 1) & 1) * (size_t)a.slots + ch.slot) * w + c] = S;
  }
}

void launch_mingru(const MinGruArgs& a, hipStream_t st) {
  if (a.n < 1) return;
  if (a.split && !a.chunks) throw std::runtime_error("mingru: chunks of a split scan are missing");
  const dim3 grid((a.w + MG_T - 1) / MG_T, a.n);
  auto go = [&](auto f32) {
    constexpr bool F32 = decltype(f32)::value;
    if (!a.chunks) {
      hipLaunchKernelGGL((mingru_kernel<F32, false, 1>), grid, dim3(MG_T), 0, st, a);
      return;
    }
    if (a.split) hipLaunchKernelGGL((mingru_kernel<F32, true, SCAN_CHUNK>), grid, dim3(MG_T), 0, st, a);
    hipLaunchKernelGGL((mingru_kernel<F32, false, SCAN_CHUNK>), grid, dim3(MG_T), 0, st, a);
  };
  if (a.f32) go(std::true_type{});
  else go(std::false_type{});
}

}  // namespace aios
