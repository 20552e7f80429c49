// Attention's partial results over key ranges (SAttnPartials), added up by whoever consumes them.
#pragma once
#include "bf16.hip.h"
#include "sigmoid_attn.h"

// Weight of every part z of head `h`, and what its sum is multiplied by: softmax parts carry their own maximum and
// sum, sigmoid parts just add and are gated.
struct PartialsHead {
    float m, mult;
};
__device__ __forceinline__ PartialsHead partials_head(const SAttnPartials& p, uint32_t h) {
    if (!p.ml) return PartialsHead{0.0f, sigmoid_f32(p.gate[h])};
    const float sink2 = p.sink[h] * 1.44269504088896340736f;
    float m = sink2;
    for (uint32_t z = 0; z < p.splits; ++z) m = fmaxf(m, p.ml[(static_cast<uint64_t>(z) * p.heads + h) * 2]);
    float l = __builtin_amdgcn_exp2f(sink2 - m);
    for (uint32_t z = 0; z < p.splits; ++z) {
        const float* const e = p.ml + (static_cast<uint64_t>(z) * p.heads + h) * 2;
        l = fmaf(e[1], __builtin_amdgcn_exp2f(e[0] - m), l);
    }
    return PartialsHead{m, 1.0f / l};
}
__device__ __forceinline__ float partials_weight(const SAttnPartials& p, const PartialsHead& e, uint32_t h, uint32_t z) {
    return p.ml ? __builtin_amdgcn_exp2f(p.ml[(static_cast<uint64_t>(z) * p.heads + h) * 2] - e.m) : 1.0f;
}
// columns c .. c + 3 (c a multiple of 4, below vdim_p) of head h
__device__ __forceinline__ f32x4 partials_sum4(const SAttnPartials& p, uint32_t h, uint32_t c) {
    const PartialsHead e = partials_head(p, h);
    const uint64_t slice = static_cast<uint64_t>(p.heads) * p.vdim_p;
    const float* const src = p.part + static_cast<uint64_t>(h) * p.vdim_p + c;
    f32x4 s{0.f, 0.f, 0.f, 0.f};
#pragma unroll 4
    for (uint32_t z = 0; z < p.splits; ++z) {
        const f32x4 v = *reinterpret_cast<const f32x4*>(src + z * slice);
        const float w = partials_weight(p, e, h, z);
        s.x = fmaf(v.x, w, s.x); s.y = fmaf(v.y, w, s.y); s.z = fmaf(v.z, w, s.z); s.w = fmaf(v.w, w, s.w);
    }
    s.x *= e.mult; s.y *= e.mult; s.z *= e.mult; s.w *= e.mult;
    return s;
}
__device__ __forceinline__ float partials_sum(const SAttnPartials& p, uint32_t h, uint32_t c) {
    const PartialsHead e = partials_head(p, h);
    float s = 0.0f;
    for (uint32_t z = 0; z < p.splits; ++z) s = fmaf(p.part[(static_cast<uint64_t>(z) * p.heads + h) * p.vdim_p + c], partials_weight(p, e, h, z), s);
    return s * e.mult;
}
