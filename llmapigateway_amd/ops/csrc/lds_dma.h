// Transfers from global memory straight to LDS, and the barriers that wait (or
// do not wait) for them.
#pragma once

#include "common.h"

// lds_barrier: LDS data of the workgroup's waves is visible after it, while
// transfers of dma16 stay in flight across it; dma_barrier: they too have
// landed.
__device__ __forceinline__ void lds_barrier() {
    asm volatile("s_waitcnt lgkmcnt(0)\n\ts_barrier" ::: "memory");
}
__device__ __forceinline__ void dma_barrier() {
    asm volatile("s_waitcnt vmcnt(0) lgkmcnt(0)\n\ts_barrier" ::: "memory");
}
// 16 bytes a lane from global memory to LDS at lds (wave-uniform) + 16*lane.
// As asm: the compiler would let every later LDS read wait for the transfer;
// here only dma_barrier does. (Wait counts it places for its own loads are
// only stricter for the transfers it does not see.)
__device__ __forceinline__ void dma16(const bf16* src, const bf16* lds) {
    const uint32_t at = __builtin_amdgcn_readfirstlane(
        (uint32_t)(uintptr_t)(const __attribute__((address_space(3))) bf16*)lds);
    asm volatile("s_mov_b32 m0, %0\n\ts_nop 0\n\tglobal_load_lds_dwordx4 %1, off"
                 ::"s"(at), "v"(src) : "memory", "m0");
}
// The same with everything but the lane's part uniform: 16 bytes a lane from
// base + offset (bytes) to LDS byte address lds + 16*lane.
__device__ __forceinline__ uint32_t lds_address(const void* p) {
    return (uint32_t)(uintptr_t)(const __attribute__((address_space(3))) char*)p;
}
__device__ __forceinline__ void dma16(const void* base, uint32_t offset, uint32_t lds) {
    asm volatile("s_mov_b32 m0, %0\n\ts_nop 0\n\tglobal_load_lds_dwordx4 %1, %2"
                 ::"s"(lds), "v"(offset), "s"(base) : "memory", "m0");
}
