// attn_lds.h — LDS-DMA staging and fragment reads shared by latent_attn.hip and window_attn.hip.
//
// The fragment reads are inline asm: hipcc cannot tell a ds_read from an LDS-DMA still in flight into another ring stage and
// would drain vmcnt in front of it.  The kernels order DMA -> read with their own counted vmcnt + barrier, and wait_lds()
// followed by an empty asm statement that names the destination orders read -> use.
#pragma once
#include "common.h"
#include <type_traits>
#include <utility>

typedef __attribute__((address_space(3))) void attn_lds_void;
typedef __attribute__((address_space(1))) const void attn_glb_void;

__device__ __forceinline__ unsigned lds_addr(const void* p) { return (unsigned)(uintptr_t)(const attn_lds_void*)p; }
// 64 lanes x 16 bytes from per-lane global addresses to 1 KiB of LDS at a wave-uniform address; AUX 2: read once (nt)
template <int AUX = 0>
__device__ __forceinline__ void lds_dma16(const void* gsrc, void* lds_wave_base) {
    __builtin_amdgcn_global_load_lds((attn_glb_void*)gsrc, (attn_lds_void*)lds_wave_base, 16, 0, AUX);
}
// 64 lanes x 4 bytes: 256 bytes of LDS
__device__ __forceinline__ void lds_dma4(const void* gsrc, void* lds_wave_base) {
    __builtin_amdgcn_global_load_lds((attn_glb_void*)gsrc, (attn_lds_void*)lds_wave_base, 4, 0, 0);
}
template <int OFF>
__device__ __forceinline__ void lds_read_b128(u32x4_t& dst, unsigned addr) {
    asm volatile("ds_read_b128 %0, %1 offset:%2" : "=v"(dst) : "v"(addr), "i"(OFF));
}
template <int OFF>
__device__ __forceinline__ void lds_read_tr16_b64(u32x2_t& dst, unsigned addr) {
    asm volatile("ds_read_b64_tr_b16 %0, %1 offset:%2" : "=v"(dst) : "v"(addr), "i"(OFF));
}
__device__ __forceinline__ void wait_lds() { asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory"); }
template <int N>
__device__ __forceinline__ void wait_vm() { asm volatile("s_waitcnt vmcnt(%0)" ::"i"(N) : "memory"); }

// 16-byte chunk permutation inside a 128-byte group of an LDS row: eight consecutive rows hit eight different chunks (row
// reads), and the four rows x two chunks of a transposed read hit eight different chunks as well
__device__ __forceinline__ int attn_swz(int row) { return ((row & 3) << 1) | ((row >> 2) & 1); }

template <int N, class F, int... I>
__device__ __forceinline__ void static_for_impl(F&& f, std::integer_sequence<int, I...>) {
    (f(std::integral_constant<int, I>{}), ...);
}
template <int N, class F>
__device__ __forceinline__ void static_for(F&& f) {
    static_for_impl<N>(f, std::make_integer_sequence<int, N>{});
}
