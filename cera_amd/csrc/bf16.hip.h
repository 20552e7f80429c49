// bfloat16 element helpers and the matrix-core operand types of the float-weight kernels.
//
// Those kernels run in one of two element types: __bf16 (matrix products and activations in
// bfloat16, accumulation in f32) and float (every product in true 32-bit on the f32 matrix cores,
// weights widened exactly).  ElemOps<T> is what differs between them below the kernel level.
#pragma once
#include "common.hip.h"

typedef __bf16 bf16x2 __attribute__((ext_vector_type(2)));
typedef __bf16 bf16x4 __attribute__((ext_vector_type(4)));
typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));
typedef float f32x4 __attribute__((ext_vector_type(4)));

__device__ __forceinline__ float bf16_lo(uint32_t pair) { return __builtin_bit_cast(float, pair << 16); }
__device__ __forceinline__ float bf16_hi(uint32_t pair) { return __builtin_bit_cast(float, pair & 0xFFFF0000u); }

// 1 / (1 + exp(-z)); exp overflowing to infinity gives 0, as it should
__device__ __forceinline__ float sigmoid_f32(float z) { return 1.0f / (1.0f + expf(-z)); }
// The same on the hardware's exponential and reciprocal (about 1 ulp each), for the inner loop of
// attention: z stays within the range in which exp2's argument is exact enough (|z| < 2^10).
__device__ __forceinline__ float sigmoid_fast(float z) {
    return __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(z * -1.44269504088896340736f));
}

template <typename T> struct ElemOps;
template <> struct ElemOps<__bf16> {
    __device__ static __forceinline__ __bf16 from(float v) { return static_cast<__bf16>(v); }
    __device__ static __forceinline__ void store4(__bf16* p, float a, float b, float c, float d) {
        *reinterpret_cast<bf16x4*>(p) = bf16x4{static_cast<__bf16>(a), static_cast<__bf16>(b), static_cast<__bf16>(c), static_cast<__bf16>(d)};
    }
    __device__ static __forceinline__ void store8(__bf16* p, const float (&v)[8]) {
        bf16x8 o;
#pragma unroll
        for (int i = 0; i < 8; ++i) o[i] = static_cast<__bf16>(v[i]);
        *reinterpret_cast<bf16x8*>(p) = o;
    }
    // acc += 8 weights (two bf16 per dword) . 8 activations
    typedef uint4 X8;
    __device__ static __forceinline__ X8 ld8(const __bf16* p) { return *reinterpret_cast<const uint4*>(p); }
    __device__ static __forceinline__ float dot8(uint4 w, X8 x, float acc) {
        acc = __builtin_amdgcn_fdot2_f32_bf16(__builtin_bit_cast(bf16x2, w.x), __builtin_bit_cast(bf16x2, x.x), acc, false);
        acc = __builtin_amdgcn_fdot2_f32_bf16(__builtin_bit_cast(bf16x2, w.y), __builtin_bit_cast(bf16x2, x.y), acc, false);
        acc = __builtin_amdgcn_fdot2_f32_bf16(__builtin_bit_cast(bf16x2, w.z), __builtin_bit_cast(bf16x2, x.z), acc, false);
        return __builtin_amdgcn_fdot2_f32_bf16(__builtin_bit_cast(bf16x2, w.w), __builtin_bit_cast(bf16x2, x.w), acc, false);
    }
};
template <> struct ElemOps<float> {
    __device__ static __forceinline__ float from(float v) { return v; }
    __device__ static __forceinline__ void store4(float* p, float a, float b, float c, float d) {
        *reinterpret_cast<float4*>(p) = make_float4(a, b, c, d);
    }
    __device__ static __forceinline__ void store8(float* p, const float (&v)[8]) {
        store4(p, v[0], v[1], v[2], v[3]);
        store4(p + 4, v[4], v[5], v[6], v[7]);
    }
    struct X8 { float4 a, b; };
    __device__ static __forceinline__ X8 ld8(const float* p) {
        return X8{reinterpret_cast<const float4*>(p)[0], reinterpret_cast<const float4*>(p)[1]};
    }
    __device__ static __forceinline__ float dot8(uint4 w, const X8& x, float acc) {
        acc = fmaf(bf16_lo(w.x), x.a.x, acc); acc = fmaf(bf16_hi(w.x), x.a.y, acc);
        acc = fmaf(bf16_lo(w.y), x.a.z, acc); acc = fmaf(bf16_hi(w.y), x.a.w, acc);
        acc = fmaf(bf16_lo(w.z), x.b.x, acc); acc = fmaf(bf16_hi(w.z), x.b.y, acc);
        acc = fmaf(bf16_lo(w.w), x.b.z, acc); return fmaf(bf16_hi(w.w), x.b.w, acc);
    }
};

// x[c .. c + 8) of a vector of n floats, zeros behind its end; whole: 16-byte aligned and in whole eights
__device__ __forceinline__ void load8(const float* x, uint32_t c, uint32_t n, bool whole, float (&v)[8]) {
    if (whole && c < n) {
        const float4 a = *reinterpret_cast<const float4*>(x + c), b = *reinterpret_cast<const float4*>(x + c + 4);
        v[0] = a.x; v[1] = a.y; v[2] = a.z; v[3] = a.w; v[4] = b.x; v[5] = b.y; v[6] = b.z; v[7] = b.w;
    } else {
#pragma unroll
        for (int i = 0; i < 8; ++i) v[i] = c + i < n ? x[c + i] : 0.0f;
    }
}
