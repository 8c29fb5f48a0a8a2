// Loads from memory straight into LDS (gfx950: 16 bytes a lane), and the waits and barriers that go with them.  The
// compiler does not know that such a load is in flight: whoever stages with it waits with `arrived` and then meets the
// block's other waves in `lds_barrier`, before anything staged is read.
#pragma once
#include "common.h"

// Lane l's 16 bytes at `src` land at LDS byte address `lds` + 16 l (`lds` is taken from the wave's first lane).
__device__ __forceinline__ void load_to_lds(const void* src, unsigned lds) {
  asm volatile("s_mov_b32 m0, %0\n\ts_nop 0\n\tglobal_load_lds_dwordx4 %1, off" ::"s"(
                   __builtin_amdgcn_readfirstlane(lds)),
               "v"(src)
               : "memory");
}

// Waits until all of this wave's loads have arrived.  (The same wait twice: the second one for the compiler's own count,
// which then knows that what it loaded itself has arrived and puts no waits for it behind later loads to LDS.)
__device__ __forceinline__ void arrived() {
  asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
  __builtin_amdgcn_s_waitcnt(0x0f70);
}

// A barrier that waits for this wave's LDS accesses and not for its loads from memory.
__device__ __forceinline__ void lds_barrier() { asm volatile("s_waitcnt lgkmcnt(0)\n\ts_barrier" ::: "memory"); }

__device__ __forceinline__ unsigned lds_address(const void* p) {
  return (unsigned)(size_t)(const __attribute__((address_space(3))) unsigned char*)p;
}
