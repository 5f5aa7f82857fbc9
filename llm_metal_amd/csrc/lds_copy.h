// Copies from memory straight into LDS for the attention kernels.
#pragma once
#include "devutil.h"

namespace lmhip {

typedef __attribute__((address_space(3))) void lds_void;

// One wave-wide copy of 1 KB from memory into LDS without passing registers: lane i's 16 bytes land at lds_base + 16 i
// (M0 holds the wave-uniform base).  Written as assembly so that the compiler does not count it among its own loads:
// it cannot tell which LDS bytes a pending copy will write and would wait for ALL copies in flight before every LDS
// read.  The kernels wait for their copies themselves, once per step (FA_WAIT_AND_BARRIER); loads retire in order, so
// a wait that the compiler inserts for a load of its own can only wait longer than it has to, never too short.
__device__ __forceinline__ void copy_to_lds_1k(const uint4 *src_lane, uint4 *lds_base)
{
    const uint32_t base = __builtin_amdgcn_readfirstlane((uint32_t)(uintptr_t)(lds_void *)lds_base);
    asm volatile("s_mov_b32 m0, %1\n\tglobal_load_lds_dwordx4 %0, off" :: "v"(src_lane), "s"(base) : "memory", "m0");
}

#define FA_WAIT_AND_BARRIER() asm volatile("s_waitcnt vmcnt(0) lgkmcnt(0)\n\ts_barrier" ::: "memory")

}  // namespace lmhip
