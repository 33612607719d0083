// 32-bit matrix product of the fp32 engines: C (+)= A x W^T with fp32 activations, bf16 weights widened
// exactly, fp32 products and sums (v_mfma_f32_16x16x4_f32: no reduced-precision mode).
#include <stdexcept>

#include "../latent.h"
#include "gemm_common.h"

namespace aios {

constexpr int GF_T = 64, GF_K = 16, GF_LD = GF_K + 1;

// rows of a grouped product (launch_gemm_f32_grouped); tiles null: plain rows
struct GroupRows {
  const int4* tiles;
  const int* n_tiles;
  const int* token;
};

// 64 x 64 tile, four waves of 32 x 32 (2 x 2 accumulators)
__global__ void __launch_bounds__(256) gemm_f32_kernel(const float* __restrict__ A, int lda, const bf16_t* __restrict__ W,
                                                       int ldw, int M, int N, int K, float* __restrict__ C, int ldc, int acc_c,
                                                       GroupRows gr) {
  __shared__ float sA[GF_T * GF_LD], sB[GF_T * GF_LD];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int r16 = lane & 15, q = lane >> 4;
  int m0 = blockIdx.y * GF_T;
  const int n0 = blockIdx.x * GF_T;
  if (gr.tiles) {
    if ((int)blockIdx.y >= *gr.n_tiles) return;
    const int4 t = gr.tiles[blockIdx.y];
    m0 = t.y;
    M = t.y + t.z;
    W += (size_t)t.x * N * ldw;
  }
  const int wm = (wave >> 1) * 32, wn = (wave & 1) * 32;
  gf32x4 acc[2][2];
#pragma unroll
  for (int i = 0; i < 2; ++i)
#pragma unroll
    for (int j = 0; j < 2; ++j) acc[i][j] = gf32x4{0.f, 0.f, 0.f, 0.f};
  const int lr = tid >> 2, lc = (tid & 3) * 4;  // this thread's row and first column of each staged tile
  const float* arow = A;
  if (m0 + lr < M) arow = A + (size_t)(gr.token ? gr.token[m0 + lr] : m0 + lr) * lda;
  for (int k0 = 0; k0 < K; k0 += GF_K) {
    float4 av = make_float4(0.f, 0.f, 0.f, 0.f);
    uint2 bv = make_uint2(0, 0);
    if (m0 + lr < M) av = *(const float4*)(arow + k0 + lc);
    if (n0 + lr < N) bv = *(const uint2*)(W + (size_t)(n0 + lr) * ldw + k0 + lc);
    __syncthreads();
    float* pa = sA + lr * GF_LD + lc;
    float* pb = sB + lr * GF_LD + lc;
    pa[0] = av.x; pa[1] = av.y; pa[2] = av.z; pa[3] = av.w;
    pb[0] = __uint_as_float(bv.x << 16); pb[1] = __uint_as_float(bv.x & 0xffff0000u);
    pb[2] = __uint_as_float(bv.y << 16); pb[3] = __uint_as_float(bv.y & 0xffff0000u);
    __syncthreads();
#pragma unroll
    for (int k = 0; k < GF_K; k += 4) {
      float af[2], bf[2];
#pragma unroll
      for (int i = 0; i < 2; ++i) {
        af[i] = sA[(wm + 16 * i + r16) * GF_LD + k + q];
        bf[i] = sB[(wn + 16 * i + r16) * GF_LD + k + q];
      }
#pragma unroll
      for (int i = 0; i < 2; ++i)
#pragma unroll
        for (int j = 0; j < 2; ++j) acc[i][j] = __builtin_amdgcn_mfma_f32_16x16x4f32(af[i], bf[j], acc[i][j], 0, 0, 0);
    }
  }
#pragma unroll
  for (int j = 0; j < 2; ++j) {
    const int n = n0 + wn + 16 * j + r16;
    if (n >= N) continue;
#pragma unroll
    for (int i = 0; i < 2; ++i)
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const int m = m0 + wm + 16 * i + 4 * q + e;
        if (m < M) {
          float* c = C + (size_t)m * ldc + n;
          *c = acc_c ? *c + acc[i][j][e] : acc[i][j][e];
        }
      }
  }
}

void launch_gemm_f32(const float* A, int lda, const bf16_t* W, int ldw, int M, int N, int K, float* C, int ldc,
                     int accumulate, hipStream_t st) {
  if (K % GF_K || lda % 4 || ldw % 4) throw std::runtime_error("gemm_f32: K must be a multiple of 16, rows 16-byte aligned");
  if (M < 1 || N < 1) return;
  hipLaunchKernelGGL(gemm_f32_kernel, dim3((N + GF_T - 1) / GF_T, (M + GF_T - 1) / GF_T), dim3(256), 0, st, A, lda, W, ldw,
                     M, N, K, C, ldc, accumulate, GroupRows{nullptr, nullptr, nullptr});
}

void launch_gemm_f32_grouped(const float* A, int lda, const int* token, const bf16_t* W, const int4* tiles, const int* n_tiles,
                             int max_tiles, int N, int K, float* C, hipStream_t st) {
  if (K % GF_K || lda % 4) throw std::runtime_error("gemm_f32: K must be a multiple of 16, rows 16-byte aligned");
  if (max_tiles < 1 || N < 1) return;
  hipLaunchKernelGGL(gemm_f32_kernel, dim3((N + GF_T - 1) / GF_T, max_tiles), dim3(256), 0, st, A, lda, W, K, 0, N, K, C, N, 0,
                     GroupRows{tiles, n_tiles, token});
}

}  // namespace aios
