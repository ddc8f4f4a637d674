// Direct global -> LDS loads (gfx950): lane i's 16 (4) bytes land at the LDS byte address `lds` + 16 i (4 i); `lds` is
// wave-uniform.  Issued as assembly: through the compiler's own builtin every LDS read that follows first waits for all such
// loads in flight, whichever buffer it reads, so a stage filled ahead would not be ahead.  The kernel waits itself, once per
// stage: wait_direct_loads() in front of the barrier.
#pragma once
#include "common.h"

SYM_DEV unsigned int lds_address(const void* p) {
  return (unsigned int)(uintptr_t)(__attribute__((address_space(3))) const char*)p;
}
SYM_DEV void direct_load16(const void* src, unsigned int lds) {
  asm volatile("s_mov_b32 m0, %0\n\tglobal_load_lds_dwordx4 %1, off" ::"s"(lds), "v"(src) : "memory", "m0");
}
SYM_DEV void direct_load4(const void* src, unsigned int lds) {
  asm volatile("s_mov_b32 m0, %0\n\tglobal_load_lds_dword %1, off" ::"s"(lds), "v"(src) : "memory", "m0");
}
// (the builtin, so that the compiler knows its own loads from before have arrived as well)
SYM_DEV void wait_direct_loads() { __builtin_amdgcn_s_waitcnt(0x0f70); }   // vmcnt(0)
