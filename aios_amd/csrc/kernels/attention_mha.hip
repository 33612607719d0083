// Causal flash attention over contiguous per-head keys and values (latent.h, expanded form): one
// sequence's T new tokens over keys [0, start + T), query-key and value dimensions of their own, an
// optional sliding window, sink logit per head (it starts the running maximum and sum: it has no key and no
// value) and output gate, and an optional rotation of part of the queries.
//
// Four waves of 32 query rows; 64-key tiles of K and V in two LDS buffers, fed by two register buffers, one
// barrier per tile -- the pipeline of the paged GQA kernel (attention_prefill.hip), whose S^T = K Q^T /
// O^T += V^T P^T arrangement it shares: a lane holds one query row's scores, and P^T goes from the score
// accumulators into the value product without leaving registers.  The softmax weights enter that product
// as two bf16 terms (hi + lo).
//
// PG: grouped-query attention over its paged cache -- a 64-key tile is one cache block -- with a soft cap and chunks.
#include <algorithm>

#include "../latent.h"
#include "gemm_common.h"

namespace aios {

typedef short mv4i16 __attribute__((ext_vector_type(4)));

constexpr int MH_KT = 64;  // keys per tile

template <int DK, int DV, bool PG>
__global__ void __launch_bounds__(256) __attribute__((amdgpu_waves_per_eu(DK + DV <= 256 ? 2 : 1))) attn_mha_kernel(MhaPrefillArgs a) {
  constexpr int KS = DK / 16, OT = DV / 32;
  constexpr int KROW = DK + 8, VROW = DV + 32;  // (conflict-free row-major and transposed reads)
  constexpr int TILE_ELEMS = MH_KT * (KROW + VROW);
  extern __shared__ __attribute__((aligned(16))) bf16_t mh_smem[];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int l32 = lane & 31, half = lane >> 5;
  // heaviest query blocks first; the second half of an even head count lightest-first, so that the two
  // workgroups that share a CU add up to the same number of tiles
  const int nx = gridDim.x, ny = gridDim.y;
  int qb, h;
  if ((ny & 1) == 0) {
    const int L = blockIdx.y * nx + blockIdx.x, W2 = nx * ny / 2;
    if (L < W2) {
      qb = nx - 1 - L % nx;
      h = L / nx;
    } else {
      qb = (L - W2) % nx;
      h = ny / 2 + (L - W2) / nx;
    }
  } else {
    qb = nx - 1 - blockIdx.x;
    h = blockIdx.y;
  }
  const int t0 = qb * 128, tq = t0 + wave * 32 + l32;
  const bool qvalid = tq < a.T;
  const int tql = qvalid ? tq : a.T - 1;
  const int qpos = a.start + tql;
  int qlow = a.window ? max(0, qpos - a.window + 1) : 0;  // first visible key
  if (PG && a.chunk) qlow = max(qlow, qpos - qpos % a.chunk);
  const uint32_t qspan = (uint32_t)(qpos - qlow);
  gbf16x8 qf[KS];
  const float sc = a.scale * 1.4426950408889634f;
  if constexpr (PG) {
    const bf16_t* qp = a.q16 + ((size_t)tql * a.H + h) * a.dkp + 8 * half;
#pragma unroll
    for (int s = 0; s < KS; ++s) {
      uint4 u = make_uint4(0, 0, 0, 0);
      if (16 * s < a.dkp) u = *(const uint4*)(qp + 16 * s);
      qf[s] = __builtin_bit_cast(gbf16x8, u);
    }
  } else {
    const float* qp = a.q + (size_t)tql * a.ldq + h * a.dkp + 8 * half;
#pragma unroll
    for (int s = 0; s < KS; ++s) {
      uint4 u = make_uint4(0, 0, 0, 0);
      if (16 * s < a.dkp) {
        float4 x0 = *(const float4*)(qp + 16 * s), x1 = *(const float4*)(qp + 16 * s + 4);
        const int i0 = 16 * s + 8 * half - a.qrot;  // place in the rotated part (eight numbers are in or out together)
        if (i0 >= 0 && i0 < a.rot) {
          const float2* cs = a.rope + (size_t)(a.pos0 + tql) * (a.rot >> 1) + (i0 >> 1);
          auto turn = [&](float& x, float& y, int i) {
            if (i0 + 2 * i >= a.rot) return;
            const float2 t = cs[i];
            const float u = x, v = y;
            x = u * t.x - v * t.y;
            y = v * t.x + u * t.y;
          };
          turn(x0.x, x0.y, 0);
          turn(x0.z, x0.w, 1);
          turn(x1.x, x1.y, 2);
          turn(x1.z, x1.w, 3);
        }
        u = make_uint4(pk_bf16(x0.x * sc, x0.y * sc), pk_bf16(x0.z * sc, x0.w * sc), pk_bf16(x1.x * sc, x1.y * sc),
                       pk_bf16(x1.z * sc, x1.w * sc));
      }
      qf[s] = __builtin_bit_cast(gbf16x8, u);
    }
  }
  gf32x16 o[OT];
#pragma unroll
  for (int i = 0; i < OT; ++i)
#pragma unroll
    for (int e = 0; e < 16; ++e) o[i][e] = 0.f;
  float m_run = a.sink ? a.sink[h] * 1.4426950408889634f : -INFINITY;
  float l_run = a.sink ? 1.f : 0.f;

  const float cap = PG ? a.softcap * 1.4426950408889634f : 0.f;
  const int last_pos = a.start + min(a.T, t0 + 128) - 1;  // highest query position of the block
  const int ntiles = last_pos / MH_KT + 1;
  int klow = a.window ? max(0, a.start + t0 - a.window + 1) : 0;  // the block's first visible key
  if (PG && a.chunk) klow = max(klow, (a.start + t0) / a.chunk * a.chunk);
  const int kt0 = klow / MH_KT;
  const int last_key = a.start + a.T - 1;
  constexpr int KP = MH_KT * DK / 8 / 256, VP = MH_KT * DV / 8 / 256;  // 16-B pieces per thread
  struct Regs {
    gu32x4 k[KP], v[VP];
  };
  const int kvh = PG ? h / (a.H / a.G) : h, ldk = PG ? a.dkp : a.ldkv, ldv = PG ? a.dvp : a.ldkv;
  const size_t belems = PG ? (size_t)a.G * MH_KT * (a.dkp + a.dvp) : 0;
  const bf16_t* kb = PG ? a.pool + (size_t)kvh * MH_KT * a.dkp : a.k + (size_t)h * a.dkp;
  const bf16_t* vb = PG ? a.pool + (size_t)a.G * MH_KT * a.dkp + (size_t)kvh * MH_KT * a.dvp : a.v + (size_t)h * a.dvp;
  int next = PG ? a.bt[min(kt0, ntiles - 1)] : 0;  // block of the tile that is requested next
  auto load = [&](Regs& r, int kt) {
    kt = min(kt, ntiles - 1);  // (the pipeline's tail requests are re-reads)
    const size_t blk = PG ? (size_t)next * belems : 0;
    if constexpr (PG) next = a.bt[min(kt + 1, ntiles - 1)];
    static_for<KP>([&](auto I) {
      constexpr int i = decltype(I)::value;
      const int idx = tid + 256 * i, c = idx % (DK / 8);
      const int key = PG ? idx / (DK / 8) : min(kt * MH_KT + idx / (DK / 8), last_key);
      r.k[i] = gu32x4{0, 0, 0, 0};
      if (c * 8 < a.dkp) r.k[i] = *(const gu32x4*)(kb + blk + (size_t)key * ldk + c * 8);
    });
    static_for<VP>([&](auto I) {
      constexpr int i = decltype(I)::value;
      const int idx = tid + 256 * i, c = idx % (DV / 8);
      const int key = PG ? idx / (DV / 8) : min(kt * MH_KT + idx / (DV / 8), last_key);
      r.v[i] = gu32x4{0, 0, 0, 0};
      if (c * 8 < a.dvp) r.v[i] = *(const gu32x4*)(vb + blk + (size_t)key * ldv + c * 8);
    });
  };
  auto stage = [&](const Regs& r, bf16_t* buf) {
    static_for<KP>([&](auto I) {
      constexpr int i = decltype(I)::value;
      const int idx = tid + 256 * i;
      *(gu32x4*)(buf + (idx / (DK / 8)) * KROW + (idx % (DK / 8)) * 8) = r.k[i];
    });
    bf16_t* sV = buf + MH_KT * KROW;
    static_for<VP>([&](auto I) {
      constexpr int i = decltype(I)::value;
      const int idx = tid + 256 * i;
      *(gu32x4*)(sV + (idx / (DV / 8)) * VROW + (idx % (DV / 8)) * 8) = r.v[i];
    });
  };
  auto math = [&](const bf16_t* sK, int kt) {
    const bf16_t* sV = sK + MH_KT * KROW;
    gf32x16 st[2];
#pragma unroll
    for (int t = 0; t < 2; ++t) {
#pragma unroll
      for (int e = 0; e < 16; ++e) st[t][e] = 0.f;
      const bf16_t* kr = sK + (t * 32 + l32) * KROW + 8 * half;
#pragma unroll
      for (int s = 0; s < KS; ++s) {
        const gbf16x8 kf = __builtin_bit_cast(gbf16x8, *(const gu32x4*)(kr + 16 * s));
        st[t] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(kf, qf[s], st[t], 0, 0, 0);
      }
    }
    const int kbase = kt * MH_KT;
    const bool full = kbase + MH_KT - 1 <= qpos && kbase >= qlow;
    const int krel = kbase + 4 * half - qlow;
    float mx = -INFINITY;
#pragma unroll
    for (int t = 0; t < 2; ++t)
#pragma unroll
      for (int r = 0; r < 16; ++r) {
        if (PG && a.softcap > 0.f)  // (the product is the exponent of tanh's exponential)
          st[t][r] = fmaf(-2.f * cap, __builtin_amdgcn_rcpf(__builtin_amdgcn_exp2f(st[t][r]) + 1.f), cap);
        // (visible: 0 <= key - qlow <= qpos - qlow, one unsigned comparison)
        if (!full && (uint32_t)(krel + t * 32 + (r & 3) + 8 * (r >> 2)) > qspan) st[t][r] = -INFINITY;
        mx = fmaxf(mx, st[t][r]);
      }
    mx = fmaxf(mx, __shfl_xor(mx, 32, 64));
    const float mn = fmaxf(m_run, mx);
    const float ms = mn == -INFINITY ? 0.f : mn;  // (no visible key yet: a window that starts in a later tile)
    const float alpha = __builtin_amdgcn_exp2f(m_run - ms);
    float ps = 0.f;
    uint32_t pb[2][8], pl[2][8];  // P^T as packed bf16 pairs (hi, lo), accumulator order
#pragma unroll
    for (int t = 0; t < 2; ++t)
#pragma unroll
      for (int r = 0; r < 16; r += 2) {
        const float p0 = __builtin_amdgcn_exp2f(st[t][r] - ms), p1 = __builtin_amdgcn_exp2f(st[t][r + 1] - ms);
        ps += p0 + p1;
        const uint32_t hi = pk_bf16(p0, p1);
        pb[t][r >> 1] = hi;
        pl[t][r >> 1] = pk_bf16(p0 - __uint_as_float(hi << 16), p1 - __uint_as_float(hi & 0xffff0000u));
      }
    ps += __shfl_xor(ps, 32, 64);
    l_run = l_run * alpha + ps;
    if (__any(mn != m_run)) {
#pragma unroll
      for (int i = 0; i < OT; ++i)
#pragma unroll
        for (int e = 0; e < 16; ++e) o[i][e] *= alpha;
    }
    m_run = mn;
    // O^T += V^T P^T: k-step s uses accumulator registers 8 (s % 2) .. + 7 of tile half s / 2, i.e. keys
    // 16 s + 4 half + {0..3} and 16 s + 8 + 4 half + {0..3}
#pragma unroll
    for (int s = 0; s < 4; ++s) {
      const int t = s >> 1, rb = (s & 1) * 4;
      const gbf16x8 pf = __builtin_bit_cast(gbf16x8, make_uint4(pb[t][rb], pb[t][rb + 1], pb[t][rb + 2], pb[t][rb + 3]));
      const gbf16x8 pg = __builtin_bit_cast(gbf16x8, make_uint4(pl[t][rb], pl[t][rb + 1], pl[t][rb + 2], pl[t][rb + 3]));
#pragma unroll
      for (int i = 0; i < OT; ++i) {
        const bf16_t* va = sV + (16 * s + 4 * half + ((lane & 15) >> 2)) * VROW + i * 32 + 16 * ((lane >> 4) & 1) +
                           4 * (lane & 3);
        const mv4i16 x0 = __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) mv4i16*)va);
        const mv4i16 x1 =
            __builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) mv4i16*)(va + 8 * VROW));
        const gbf16x8 vf = __builtin_bit_cast(gbf16x8, __builtin_shufflevector(x0, x1, 0, 1, 2, 3, 4, 5, 6, 7));
        o[i] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(vf, pf, o[i], 0, 0, 0);
        o[i] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(vf, pg, o[i], 0, 0, 0);
      }
    }
  };
  bf16_t* L0 = mh_smem;
  bf16_t* L1 = mh_smem + TILE_ELEMS;
  Regs A, B;
  load(A, kt0);
  load(B, kt0 + 1);
  stage(A, L0);
  __syncthreads();
  for (int kt = kt0; kt < ntiles; kt += 2) {  // (an odd count computes one fully masked pad tile)
    load(A, kt + 2);
    math(L0, kt);
    stage(B, L1);
    __syncthreads();
    load(B, kt + 3);
    math(L1, kt + 1);
    stage(A, L0);
    __syncthreads();
  }
  if (!qvalid) return;
  const float inv = (PG ? a.out_scale : 1.f) / l_run;
  bf16_t* op = a.out + (size_t)tq * a.ldo + (size_t)h * a.dvp;
  const float* gp = a.gate ? a.gate + (size_t)tq * a.ldq + (a.head_gate ? h : (size_t)h * a.dvp) : nullptr;
#pragma unroll
  for (int i = 0; i < OT; ++i)
#pragma unroll
    for (int r = 0; r < 16; r += 4) {
      const int d = i * 32 + 8 * (r >> 2) + 4 * half;
      if (i * 32 < a.dvp) {
        float v[4];
#pragma unroll
        for (int e = 0; e < 4; ++e) v[e] = o[i][r + e] * inv;
        if (gp) {
          const float4 g = a.head_gate ? make_float4(gp[0], gp[0], gp[0], gp[0]) : *(const float4*)(gp + d);
          v[0] *= 1.f / (1.f + __expf(-g.x));
          v[1] *= 1.f / (1.f + __expf(-g.y));
          v[2] *= 1.f / (1.f + __expf(-g.z));
          v[3] *= 1.f / (1.f + __expf(-g.w));
        }
        *(uint2*)(op + d) = make_uint2(pk_bf16(v[0], v[1]), pk_bf16(v[2], v[3]));
      }
    }
}

bool mha_prefill_supports(int dkp, int dvp) {
  return dkp > 0 && dvp > 0 && dkp <= 256 && dvp <= 256 && dkp % 32 == 0 && dvp % 32 == 0;
}

template <int DK, int DV, bool PG>
static void mha_go(const MhaPrefillArgs& a, hipStream_t st) {
  constexpr size_t lds = (size_t)2 * MH_KT * ((DK + 8) + (DV + 32)) * sizeof(bf16_t);
  static_assert(lds <= 160 * 1024, "LDS");
  hipLaunchKernelGGL((attn_mha_kernel<DK, DV, PG>), dim3((a.T + 127) / 128, a.H), dim3(256), lds, st, a);
}
template <int DK, bool PG>
static void mha_dv(const MhaPrefillArgs& a, hipStream_t st) {
  if (a.dvp <= 64) mha_go<DK, 64, PG>(a, st);
  else if (a.dvp <= 128) mha_go<DK, 128, PG>(a, st);
  else mha_go<DK, 256, PG>(a, st);
}
template <bool PG>
static void mha_dk(const MhaPrefillArgs& a, hipStream_t st) {
  if (a.dkp <= 64) mha_dv<64, PG>(a, st);
  else if (a.dkp <= 128) mha_dv<128, PG>(a, st);
  else if (a.dkp <= 192) mha_dv<192, PG>(a, st);
  else mha_dv<256, PG>(a, st);
}

void launch_mha_prefill(const MhaPrefillArgs& a, hipStream_t st) {
  if (!mha_prefill_supports(a.dkp, a.dvp)) throw std::runtime_error("mha_prefill: unsupported head dimensions");
  if (a.rot % 2 || a.qrot % 8) throw std::runtime_error("mha_prefill: bad rotated part");
  if (a.pool ? a.H % std::max(1, a.G) || !a.q16 || !a.bt || a.rot || a.ldo % 4 || (a.gate && !a.head_gate)
             : a.ldkv % 8 || a.ldq % 4 || a.ldo % 4)
    throw std::runtime_error("mha_prefill: misaligned rows");
  if (a.T < 1) return;
  if (a.pool) mha_dk<true>(a, st);
  else mha_dk<false>(a, st);
}

}  // namespace aios
