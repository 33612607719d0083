// Global memory to LDS without registers in between, and the waits that order it (prefill GEMMs, gated delta rule).
#pragma once
#include "../common.h"

namespace aios {

__device__ __forceinline__ void pf_barrier() {
  asm volatile("" ::: "memory");
  __builtin_amdgcn_s_barrier();
  asm volatile("" ::: "memory");
}
template <int N>
__device__ __forceinline__ void pf_vmcnt() {
  static_assert(N >= 0 && N <= 63, "vmcnt immediate");
  asm volatile("s_waitcnt vmcnt(%0)" ::"n"(N) : "memory");
}

// LDS-DMA through inline asm: hipcc's waitcnt pass then does not see the DMA, so it no longer puts
// an `s_waitcnt vmcnt(0)` in front of the first ds_read after every issue (it cannot prove the read
// misses the DMA's target slot -- measured: that drain serialised every K-step).  The counted
// pf_vmcnt waits are the only ordering these loads need.  M0 is set and restored inside the
// statement.
__device__ __forceinline__ uint32_t pf_lds_addr(const uint8_t* p) {
  return (uint32_t)(uintptr_t)(const __attribute__((address_space(3))) uint8_t*)p;
}
__device__ __forceinline__ void pf_glds16(const void* src, uint32_t lds) {
  uint32_t keep;
  asm volatile("s_mov_b32 %0, m0\n\ts_mov_b32 m0, %2\n\ts_nop 0\n\tglobal_load_lds_dwordx4 %1, off\n\ts_mov_b32 m0, %0"
               : "=&s"(keep)
               : "v"(src), "s"(lds)
               : "memory");
}
__device__ __forceinline__ void pf_glds4(const void* src, uint32_t lds) {
  uint32_t keep;
  asm volatile("s_mov_b32 %0, m0\n\ts_mov_b32 m0, %2\n\ts_nop 0\n\tglobal_load_lds_dword %1, off\n\ts_mov_b32 m0, %0"
               : "=&s"(keep)
               : "v"(src), "s"(lds)
               : "memory");
}

}  // namespace aios
