// LDS-DMA helpers (gfx950): global -> LDS copies that bypass the VGPRs, with hand-counted completion.
#pragma once
#include "common.h"

namespace nls_dma {

// LDS byte address of a pointer into the dynamic LDS array
DEVI uint32_t lds_addr(const void* p) {
  return (uint32_t)(uintptr_t)(const __attribute__((address_space(3))) void*)p;
}
// 16 B per lane global -> LDS (dst = wave-uniform `lds_dst` + 16 * lane). Inline asm: invisible to
// hipcc's waitcnt pass (no vmcnt(0) before every ds_read); completion is counted by hand.
DEVI void glds16(const void* gsrc, uint32_t lds_dst) {
  uint32_t keep;
  asm volatile("s_mov_b32 %0, m0\n\ts_mov_b32 m0, %2\n\ts_nop 0\n\tglobal_load_lds_dwordx4 %1, off\n\ts_mov_b32 m0, %0"
               : "=&s"(keep)
               : "v"(gsrc), "s"(lds_dst)
               : "memory");
}
// the same from a wave-uniform base and a byte offset per lane
DEVI void glds16(const void* base, uint32_t offset, uint32_t lds_dst) {
  uint32_t keep;
  asm volatile("s_mov_b32 %0, m0\n\ts_mov_b32 m0, %3\n\ts_nop 0\n\tglobal_load_lds_dwordx4 %1, %2\n\ts_mov_b32 m0, %0"
               : "=&s"(keep)
               : "v"(offset), "s"(base), "s"(lds_dst)
               : "memory");
}
template <int N>
DEVI void wait_vm_lgkm0() {
  asm volatile("s_waitcnt vmcnt(%0) lgkmcnt(0)" ::"i"(N) : "memory");
}

}  // namespace nls_dma
