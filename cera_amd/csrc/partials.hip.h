// Attention's partial results over key ranges (SAttnPartials), added up by whoever consumes them.
#pragma once
#include "bf16.hip.h"
#include "sigmoid_attn.h"

// Weights of the parts of heads h0 .. h0 + n - 1 into wz [n][splits], a head per thread: softmax parts carry their own
// maximum and sum, sigmoid parts just add and are gated.  The caller puts a barrier behind it.
__device__ __forceinline__ void partials_weights(const SAttnPartials& p, uint32_t h0, uint32_t n, uint32_t thread, uint32_t threads, float* wz) {
    for (uint32_t i = thread; i < n; i += threads) {
        const uint32_t h = h0 + i;
        float* const w = wz + i * p.splits;
        if (!p.ml) {
            const float g = sigmoid_f32(p.gate[h]);
            for (uint32_t z = 0; z < p.splits; ++z) w[z] = g;
            continue;
        }
        const float sink2 = p.sink[h] * 1.44269504088896340736f;
        const float2* const ml = reinterpret_cast<const float2*>(p.ml) + h;
        float m = sink2;
#pragma unroll 8
        for (uint32_t z = 0; z < p.splits; ++z) m = fmaxf(m, ml[z * p.heads].x);
        float l = __builtin_amdgcn_exp2f(sink2 - m);
#pragma unroll 8
        for (uint32_t z = 0; z < p.splits; ++z) {
            const float2 e = ml[z * p.heads];
            w[z] = __builtin_amdgcn_exp2f(e.x - m);
            l = fmaf(e.y, w[z], l);
        }
        const float inv = 1.0f / l;
        for (uint32_t z = 0; z < p.splits; ++z) w[z] *= inv;
    }
}
// columns c .. c + 3 (c a multiple of 4, below vdim_p) of head h; wz: the head's weights
__device__ __forceinline__ f32x4 partials_sum4(const SAttnPartials& p, const float* wz, uint32_t h, uint32_t c) {
    const uint64_t slice = static_cast<uint64_t>(p.heads) * p.vdim_p;
    const float* const src = p.part + static_cast<uint64_t>(h) * p.vdim_p + c;
    f32x4 s{0.f, 0.f, 0.f, 0.f};
#pragma unroll 8
    for (uint32_t z = 0; z < p.splits; ++z) {
        const f32x4 v = *reinterpret_cast<const f32x4*>(src + z * slice);
        s.x = fmaf(v.x, wz[z], s.x); s.y = fmaf(v.y, wz[z], s.y); s.z = fmaf(v.z, wz[z], s.z); s.w = fmaf(v.w, wz[z], s.w);
    }
    return s;
}
__device__ __forceinline__ float partials_sum(const SAttnPartials& p, const float* wz, uint32_t h, uint32_t c) {
    float s = 0.0f;
    for (uint32_t z = 0; z < p.splits; ++z) s = fmaf(p.part[(static_cast<uint64_t>(z) * p.heads + h) * p.vdim_p + c], wz[z], s);
    return s;
}
