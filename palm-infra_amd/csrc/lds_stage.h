// Rows straight from memory into LDS, for kernels that walk over K through a ring of stages: 16 bytes a lane and instruction,
// a wave's instruction filling 1 KB from `lds_base` on, and the wait for all but the youngest of them.
#pragma once
#include "common.h"

__device__ __forceinline__ void row_chunk_into_lds(const void* from, uint32_t lds_base) {
    asm volatile("s_mov_b32 m0, %1\n\ts_nop 0\n\tglobal_load_lds_dwordx4 %0, off" : : "v"(from), "s"(lds_base) : "m0", "memory");
}
// s_waitcnt vmcnt(N): loads come back in order, so "all but the N youngest" is a stage's rows with the later stages'
// still on their way.  (vmcnt is six bits: the low four in bits 0..3, the high two in bits 14..15.)
template <int N> __device__ __forceinline__ void all_but_the_youngest_have_arrived() {
    static_assert(N >= 0 && N < 64, "vmcnt has six bits");
    __builtin_amdgcn_s_waitcnt(0x0F70 | (N & 15) | ((N >> 4) << 14));
}
