// Attention's partial results over key ranges (SAttnPartials), added up by whoever consumes them.
#pragma once
#include "bf16.hip.h"
#include "sigmoid_attn.h"

// over each 16-lane row; every lane of a row ends up with its row's maximum
__device__ __forceinline__ float wave_row_max(float v) {
    v = fmaxf(v, dpp_f<0xB1>(v));
    v = fmaxf(v, dpp_f<0x4E>(v));
    v = fmaxf(v, dpp_f<0x141>(v));
    return fmaxf(v, dpp_f<0x140>(v));
}
// Weights of the parts of heads h0 .. h0 + n - 1 into wz [n][splits], sixteen threads per head (`threads` a multiple of
// 64, all of them call): softmax parts carry their own maximum and sum, sigmoid parts just add and are gated.  The
// caller puts a barrier behind it.
__device__ __forceinline__ void partials_weights(const SAttnPartials& p, uint32_t h0, uint32_t n, uint32_t thread, uint32_t threads, float* wz) {
    const uint32_t l16 = thread & 15;
    for (uint32_t i = thread >> 4; i < n; i += threads >> 4) {
        const uint32_t h = h0 + i;
        float* const w = wz + i * p.splits;
        if (!p.ml) {
            const float g = sigmoid_f32(p.gate[h]);
            for (uint32_t z = l16; z < p.splits; z += 16) w[z] = g;
            continue;
        }
        const float sink2 = p.sink[h] * 1.44269504088896340736f;
        const float2* const ml = reinterpret_cast<const float2*>(p.ml) + h;
        float m = sink2, l = 0.0f;
        for (uint32_t z = l16; z < p.splits; z += 16) m = fmaxf(m, ml[z * p.heads].x);
        m = wave_row_max(m);
        for (uint32_t z = l16; z < p.splits; z += 16) {
            const float2 e = ml[z * p.heads];
            w[z] = __builtin_amdgcn_exp2f(e.x - m);
            l = fmaf(e.y, w[z], l);
        }
        const float inv = 1.0f / (wave_row_sum(l) + __builtin_amdgcn_exp2f(sink2 - m));
        for (uint32_t z = l16; z < p.splits; z += 16) w[z] *= inv;
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
