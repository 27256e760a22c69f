// What the matrix-core products' tile loops and epilogues share (gemm_mfma.hip, expert_gemm.hip).
#pragma once
#include "gemm.h"

#include <type_traits>

typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));
typedef __bf16 bf16x4 __attribute__((ext_vector_type(4)));
typedef float f32x4 __attribute__((ext_vector_type(4)));
typedef float f32x16 __attribute__((ext_vector_type(16)));

template <int I, int N, class F>
__device__ __forceinline__ void static_for(F&& f) {
    if constexpr (I < N) {
        f(std::integral_constant<int, I>{});
        static_for<I + 1, N>(f);
    }
}

typedef __bf16 bf16x2 __attribute__((ext_vector_type(2)));
// The value the neighbouring lane (lane ^ 1) passes: a DPP move within each group of four lanes, no LDS.
__device__ __forceinline__ float swap_neighbours(float x) {
    int u = __float_as_int(x);
    return __int_as_float(__builtin_amdgcn_update_dpp(u, u, 0xB1, 0xf, 0xf, true));     // quad_perm [1, 0, 3, 2]
}
// x / (1 + exp(-x)) with the device's exponential and reciprocal instructions (each within an ulp; the result is
// rounded to bfloat16 right after).  For the epilogues that finish thousands of values per wave.
__device__ __forceinline__ float silu_fast_f32(float x) {
    return x * __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(x * -1.44269504088896341f));
}
// The tile loops' barrier: this wave's LDS reads and writes are done, then every wave of the block
// has arrived.  Unlike __syncthreads() it does not wait for loads from memory that are still in
// flight (the later tiles of a pipeline); the "memory" clobber keeps the compiler from moving
// memory accesses across it.
__device__ __forceinline__ void block_sync_lds() { asm volatile("s_waitcnt lgkmcnt(0)\n\ts_barrier" ::: "memory"); }

// All but the last N_ of this wave's vector memory operations have completed (they complete in order).
template <int N_>
__device__ __forceinline__ void wait_vmcnt() {
    static_assert(N_ >= 0 && N_ < 64, "vmcnt is a 6-bit counter");
    __builtin_amdgcn_s_waitcnt((N_ & 15) | (7 << 4) | (15 << 8) | ((N_ >> 4) << 14));
}
