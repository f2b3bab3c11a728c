// hybrid_common.h — helpers shared by the hybrid-decoder kernels (csrc/hybrid/*.hip).
//
// Every kernel is instantiated for two activation element types: bfloat16 travelling as raw 16-bit words
// (uint16_t, as in csrc/kernels) and float.  Whatever the activation type, residual stream, norms, recurrent state,
// gates, router and attention scores are float.
#pragma once
#include "chronos_hip.h"

namespace chronos {
namespace hy {

template <typename T> __device__ __forceinline__ float ld(const T* p);
template <> __device__ __forceinline__ float ld<float>(const float* p) { return *p; }
template <> __device__ __forceinline__ float ld<uint16_t>(const uint16_t* p) { return bf2f(*p); }
template <typename T> __device__ __forceinline__ void st(T* p, float v);
template <> __device__ __forceinline__ void st<float>(float* p, float v) { *p = v; }
template <> __device__ __forceinline__ void st<uint16_t>(uint16_t* p, float v) { *p = f2bf(v); }

// round a float through the activation type (what a value stored and read back would be)
template <typename T> __device__ __forceinline__ float rnd(float v);
template <> __device__ __forceinline__ float rnd<float>(float v) { return v; }
template <> __device__ __forceinline__ float rnd<uint16_t>(float v) { return bf2f(f2bf(v)); }

__device__ __forceinline__ float sigmoidf_(float z) { return 1.f / (1.f + expf(-z)); }
// log(sigmoid(z)) without overflow on either side
__device__ __forceinline__ float logsigmoidf_(float z) { return fminf(z, 0.f) - log1pf(expf(-fabsf(z))); }

// Transposing LDS read (gfx950): the 16 lanes of a lane group name the 8-byte pieces of a 4 x 16 matrix of 16-bit
// elements, row by row (lane l: row l / 4, columns 4 (l % 4) ..), and lane l receives column l, its 4 rows in order.
// Rows may lie anywhere.  A row-major tile thus serves as either operand of a matrix product.
__device__ __forceinline__ bf16x4 lds_read_tr4(const void* p) {
    typedef __attribute__((address_space(3))) bf16x4 lds_bf16x4;
    return __builtin_amdgcn_ds_read_tr16_b64_v4bf16((lds_bf16x4*)p);
}

__device__ __forceinline__ f32x4 mfma_16x16x16(bf16x4 a, bf16x4 b, f32x4 c) {
    typedef short s16x4 __attribute__((ext_vector_type(4)));
    return __builtin_amdgcn_mfma_f32_16x16x16bf16_1k(__builtin_bit_cast(s16x4, a), __builtin_bit_cast(s16x4, b), c, 0, 0, 0);
}

// One 1 KiB piece from memory straight into LDS: lane l's 16 bytes from its own address to LDS offset lds + 16 l (lds the
// same in all lanes).  Inline asm, so that the compiler does not wait for it before every LDS read; the kernel waits with
// dma_wait() in front of the barrier that hands the piece over.
__device__ __forceinline__ void dma_1k(const void* src, uint32_t lds) {
    asm volatile("s_mov_b32 m0, %1\n\ts_nop 0\n\tglobal_load_lds_dwordx4 %0, off" ::"v"(src), "s"(lds) : "memory");
}
__device__ __forceinline__ void dma_wait() { asm volatile("s_waitcnt vmcnt(0)" ::: "memory"); }
__device__ __forceinline__ uint32_t lds_offset(const void* p) {
    typedef __attribute__((address_space(3))) const void* lds_ptr;
    return (uint32_t)(uintptr_t)(lds_ptr)p;
}
// Piece j of a tile of rows: an LDS image of row-major rows, each CPR chunks of 16 bytes of which the last is padding
// (it spreads the rows over the banks; like the chunks past the row's n real ones it receives a copy of the last real
// one).  rows: element offset factor of each row of the tile; width: elements per row in memory.
template <int CPR> __device__ __forceinline__ void dma_rows(const uint16_t* src, const int* rows, int width, int n, int j,
                                                            uint32_t lds, int lane) {
    const int i = j * 64 + lane, row = i / CPR, ch = i - row * CPR;
    dma_1k(src + (int64_t)rows[row] * width + min(ch, n - 1) * 8, __builtin_amdgcn_readfirstlane(lds + j * 1024));
}

constexpr int kActRelu2 = 0, kActGelu = 1;
__device__ __forceinline__ float act_apply(float z, int kind) {
    if (kind == kActRelu2) {
        const float r = fmaxf(z, 0.f);
        return r * r;
    }
    return 0.5f * z * (1.f + erff(z * 0.70710678118654752440f));
}

}  // namespace hy
}  // namespace chronos
