// Shared by the kernels of libtrimkv_hybrid.so: element access by type, wavefront sums, exact splits of fp32 operands.
#pragma once

#include "common.hip.h"
#include "trimkv_hybrid.h"

namespace trimkv {

struct bf16_t { uint16_t bits; };

__device__ __forceinline__ float ld(const float* p) { return *p; }
__device__ __forceinline__ float ld(const bf16_t* p) { return bf16_bits_to_f32(p->bits); }
__device__ __forceinline__ void st(float* p, float f) { *p = f; }
__device__ __forceinline__ void st(bf16_t* p, float f) { p->bits = f32_to_bf16_bits(f); }

// four consecutive elements (16 bytes of fp32, 8 of bf16; the pointer is aligned to that)
__device__ __forceinline__ float4 ld4(const float* p) { return *(const float4*)p; }
__device__ __forceinline__ float4 ld4(const bf16_t* p) {
    const uint2 u = *(const uint2*)p;
    return make_float4(__uint_as_float(u.x << 16), __uint_as_float(u.x & 0xffff0000u), __uint_as_float(u.y << 16), __uint_as_float(u.y & 0xffff0000u));
}
__device__ __forceinline__ void st4(float* p, float4 f) { *(float4*)p = f; }
__device__ __forceinline__ void st4(bf16_t* p, float4 f) {
    uint2 u;
    u.x = (uint32_t)f32_to_bf16_bits(f.x) | ((uint32_t)f32_to_bf16_bits(f.y) << 16);
    u.y = (uint32_t)f32_to_bf16_bits(f.z) | ((uint32_t)f32_to_bf16_bits(f.w) << 16);
    *(uint2*)p = u;
}

__device__ __forceinline__ float sigmoid_f(float x) { return 1.0f / (1.0f + expf(-x)); }
// for output gates: hardware exponential and reciprocal, a few ulp
__device__ __forceinline__ float sigmoid_fast(float x) { return __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(x * -1.4426950408889634f)); }
// log(sigmoid(x)) with the library's exp and log1p
__device__ __forceinline__ float log_sigmoid_exact(float x) { return fminf(x, 0.0f) - log1pf(expf(-fabsf(x))); }

__device__ __forceinline__ float wave_sum_f(float v) {
#pragma unroll
    for (int d = 32; d > 0; d >>= 1) v += __shfl_xor(v, d, 64);
    return v;
}
__device__ __forceinline__ float wave_max_f(float v) {
#pragma unroll
    for (int d = 32; d > 0; d >>= 1) v = fmaxf(v, __shfl_xor(v, d, 64));
    return v;
}
// sum over a workgroup of `waves` wavefronts; `part` holds one float per wavefront.  Ends with every thread holding the sum;
// the caller puts a barrier in front of the next use of `part`.
__device__ __forceinline__ float block_sum_f(float v, float* part, int waves) {
    v = wave_sum_f(v);
    if ((threadIdx.x & 63) == 0) part[threadIdx.x >> 6] = v;
    __syncthreads();
    float s = 0.0f;
    for (int w = 0; w < waves; ++w) s += part[w];
    return s;
}

typedef __bf16 hy_bf16x8 __attribute__((ext_vector_type(8)));
typedef __bf16 hy_bf16x2 __attribute__((ext_vector_type(2)));
typedef float hy_f32x2 __attribute__((ext_vector_type(2)));
typedef float hy_f32x4 __attribute__((ext_vector_type(4)));
typedef float hy_f32x16 __attribute__((ext_vector_type(16)));
typedef short hy_s16x4 __attribute__((ext_vector_type(4)));
typedef uint32_t hy_u32x2 __attribute__((ext_vector_type(2)));
typedef uint32_t hy_u32x4 __attribute__((ext_vector_type(4)));
#define HY_LDS __attribute__((address_space(3)))

__device__ __forceinline__ uint32_t pack2(float lo, float hi) {
    const hy_f32x2 f = {lo, hi};
    return __builtin_bit_cast(uint32_t, __builtin_convertvector(f, hy_bf16x2));
}
// A pair of fp32 values as sums of TERMS bf16 values each: three terms carry all 24 mantissa bits, so that products with
// exact bf16 operands on the matrix cores are fp32 products; two terms carry 17 bits.
template <int TERMS>
__device__ __forceinline__ void split2(float a, float b, uint32_t (&out)[TERMS]) {
#pragma unroll
    for (int i = 0; i < TERMS; ++i) {
        const uint32_t p = pack2(a, b);
        out[i] = p;
        if (i + 1 < TERMS) {
            a -= __uint_as_float(p << 16);
            b -= __uint_as_float(p & 0xffff0000u);
        }
    }
}

__device__ __forceinline__ hy_f32x4 mfma16(hy_bf16x8 a, hy_bf16x8 b, hy_f32x4 c) { return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, c, 0, 0, 0); }
__device__ __forceinline__ hy_f32x16 mfma32(hy_bf16x8 a, hy_bf16x8 b, hy_f32x16 c) { return __builtin_amdgcn_mfma_f32_32x32x16_bf16(a, b, c, 0, 0, 0); }

// One LDS-direct load of 16 bytes per lane: lane l's bytes land at lds_addr + 16 l (lds_addr wavefront-uniform).  The compiler
// neither counts nor waits for these loads: whoever reads the LDS waits with an explicit s_waitcnt first.
__device__ __forceinline__ void load_to_lds16(const void* src, uint32_t lds_addr) {
    uint32_t saved;
    asm volatile("s_mov_b32 %0, m0\n\ts_mov_b32 m0, %2\n\ts_nop 0\n\tglobal_load_lds_dwordx4 %1, off\n\ts_mov_b32 m0, %0"
                 : "=&s"(saved) : "v"(src), "s"(lds_addr) : "memory");
}

// the same from a wavefront-uniform base and a per-lane byte offset
__device__ __forceinline__ void load_to_lds16_at(const char* base, uint32_t offset, uint32_t lds_addr) {
    uint32_t saved;
    asm volatile("s_mov_b32 %0, m0\n\ts_mov_b32 m0, %3\n\ts_nop 0\n\tglobal_load_lds_dwordx4 %1, %2\n\ts_mov_b32 m0, %0"
                 : "=&s"(saved) : "v"(offset), "s"(base), "s"(lds_addr) : "memory");
}

// The slot of a token in a window ring: the first `keep` positions own their slots, later ones take turns on `size` slots.
__device__ __forceinline__ int ring_slot(int pos, int keep, int size) { return pos < keep ? pos : keep + (pos - keep) % size; }
// The position a ring slot holds after `total` tokens (total > slot): the newest one that maps to it.
__device__ __forceinline__ int ring_position(int slot, int total, int keep, int size) {
    return slot < keep ? slot : slot + size * ((total - 1 - slot) / size);
}

// Expand a launch over the element type of activations and weights.
#define HY_BY_DTYPE(dt, T, ...)                                        \
    do {                                                               \
        if ((dt) == TRIMKV_BF16) { using T = bf16_t; __VA_ARGS__; }    \
        else { using T = float; __VA_ARGS__; }                         \
    } while (0)
#define HY_CHECK_DTYPE(fn, dt) \
    if ((dt) != TRIMKV_BF16 && (dt) != TRIMKV_F32) return fail(TRIMKV_ERR_DTYPE, "%s: dtype must be f32 or bf16 (dtype=%d)", fn, dt)

}  // namespace trimkv
