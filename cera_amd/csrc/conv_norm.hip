// Kernels of conv_norm.h.  Everything here is f32 up to the store of an output row.
#include <algorithm>

#include "bf16.hip.h"
#include "conv_norm.h"

namespace {

__device__ __forceinline__ float bf16_at(const uint16_t* p, uint64_t i) { return __builtin_bit_cast(float, static_cast<uint32_t>(p[i]) << 16); }

__global__ __launch_bounds__(256) void embed_pos_kernel(const uint16_t* __restrict__ embed, const uint16_t* __restrict__ pos,
                                                        const uint32_t* __restrict__ tokens, uint32_t token, uint32_t start,
                                                        uint32_t width, uint64_t ld, float* __restrict__ x, float* __restrict__ x0) {
    const uint32_t t = blockIdx.y, c = blockIdx.x * 256 + threadIdx.x;
    if (c >= ld) return;
    const uint64_t tok = tokens ? tokens[t] : token;
    const float v = c < width ? bf16_at(embed, tok * width + c) + bf16_at(pos, static_cast<uint64_t>(start + t) * width + c) : 0.0f;
    x[t * ld + c] = v;
    x0[t * ld + c] = v;
}

__global__ __launch_bounds__(256) void embed_streams_kernel(const uint16_t* __restrict__ embed, const uint32_t* __restrict__ tokens, uint32_t token,
                                                            uint32_t width, uint64_t ld, float* __restrict__ x, uint32_t streams, uint64_t stride,
                                                            float u_scale, float* __restrict__ u) {
    const uint32_t t = blockIdx.y, c = (blockIdx.x * 256 + threadIdx.x) * 4;   // ld is a multiple of 4
    if (c >= ld) return;
    const uint16_t* const row = embed + static_cast<uint64_t>(tokens ? tokens[t] : token) * width;
    const float4 v = make_float4(c < width ? bf16_at(row, c) : 0.0f, c + 1 < width ? bf16_at(row, c + 1) : 0.0f,
                                 c + 2 < width ? bf16_at(row, c + 2) : 0.0f, c + 3 < width ? bf16_at(row, c + 3) : 0.0f);
    for (uint32_t s = 0; s < streams; ++s) *reinterpret_cast<float4*>(x + s * stride + t * ld + c) = v;
    *reinterpret_cast<float4*>(u + t * ld + c) = make_float4(u_scale * v.x, u_scale * v.y, u_scale * v.z, u_scale * v.w);
}

// A workgroup takes `rows` consecutive rows: first 1 / rms of those rows and of the taps - 1 before them
// (recomputed, so that workgroups need nothing from each other), one row per wavefront; then the channels,
// four per thread, walking down the rows.  TAPS > 0: the window of rows and the taps' weights stay in
// registers; 0: any number of taps, re-reading the window.
constexpr int NC_WAVES = 16, NC_MAX_ROWS = 16;
__device__ __forceinline__ void fma4(float4& y, const float4& k, const float4& g) {
    y.x = fmaf(k.x, g.x, y.x); y.y = fmaf(k.y, g.y, y.y); y.z = fmaf(k.z, g.z, y.z); y.w = fmaf(k.w, g.w, y.w);
}
template <typename T, int TAPS>
__global__ __launch_bounds__(NC_WAVES * 64) void norm_conv_kernel(NormConv a, int rows) {
    __shared__ float inv[NC_MAX_ROWS + CONV_MAX_TAPS];
    const uint32_t lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    const int taps = TAPS ? TAPS : static_cast<int>(a.taps), back = taps ? taps - 1 : 0;
    const int t0 = static_cast<int>(blockIdx.x) * rows, t_end = min(t0 + rows, static_cast<int>(a.n));
    for (int t = t0 - back + static_cast<int>(wave); t < t_end; t += NC_WAVES) {
        if (t < 0) continue;
        const float* const row = a.x + static_cast<uint64_t>(t) * a.ld;
        float ss = 0.0f;
        for (uint32_t c = lane * 4; c < a.ld; c += 256) {
            const float4 v = *reinterpret_cast<const float4*>(row + c);
            ss = fmaf(v.x, v.x, ss); ss = fmaf(v.y, v.y, ss); ss = fmaf(v.z, v.z, ss); ss = fmaf(v.w, v.w, ss);
        }
        ss = wave_sum(ss);
        const float r = 1.0f / sqrtf(ss / static_cast<float>(a.width) + a.eps);
        if (lane == 0) {
            inv[t - t0 + back] = r;
            if (a.inv && t >= t0) a.inv[t] = r;
        }
    }
    __syncthreads();
    for (uint32_t c = threadIdx.x * 4; c < a.ld; c += NC_WAVES * 256) {
        const float4 w = *reinterpret_cast<const float4*>(a.w + c);
        auto h_at = [&](int t) -> float4 {
            if (t < 0) {
                const int64_t p = static_cast<int64_t>(a.start) + t;
                if (p < 0) return make_float4(0.f, 0.f, 0.f, 0.f);
                return *reinterpret_cast<const float4*>(a.ring.rows + static_cast<uint64_t>(p & (a.ring.depth - 1)) * a.ring.ld + c);
            }
            const float4 v = *reinterpret_cast<const float4*>(a.x + static_cast<uint64_t>(t) * a.ld + c);
            const float s = inv[t - t0 + back];
            return make_float4(v.x * s * w.x, v.y * s * w.y, v.z * s * w.z, v.w * s * w.w);
        };
        auto store = [&](int t, const float4& ya, const float4& yb) {
            const uint64_t at = static_cast<uint64_t>(t) * a.ld + c;
            ElemOps<T>::store4(static_cast<T*>(a.out_a) + at, ya.x, ya.y, ya.z, ya.w);
            if (a.out_b) ElemOps<T>::store4(static_cast<T*>(a.out_b) + at, yb.x, yb.y, yb.z, yb.w);
        };
        if constexpr (TAPS > 0) {
            float4 ka[TAPS], kb[TAPS], h[TAPS];
#pragma unroll
            for (int j = 0; j < TAPS; ++j) {
                ka[j] = *reinterpret_cast<const float4*>(a.wa + static_cast<uint64_t>(j) * a.ld + c);
                kb[j] = a.wb ? *reinterpret_cast<const float4*>(a.wb + static_cast<uint64_t>(j) * a.ld + c) : make_float4(0.f, 0.f, 0.f, 0.f);
            }
#pragma unroll
            for (int j = 0; j + 1 < TAPS; ++j) h[j + 1] = h_at(t0 - back + j);
            for (int t = t0; t < t_end; ++t) {
#pragma unroll
                for (int j = 0; j + 1 < TAPS; ++j) h[j] = h[j + 1];
                h[TAPS - 1] = h_at(t);
                float4 ya = h[TAPS - 1], yb = ya;
#pragma unroll
                for (int j = 0; j < TAPS; ++j) {
                    fma4(ya, ka[j], h[j]);
                    fma4(yb, kb[j], h[j]);
                }
                store(t, ya, yb);
            }
        } else {
            for (int t = t0; t < t_end; ++t) {
                const float4 h = h_at(t);
                float4 ya = h, yb = h;
                for (int j = 0; j < taps; ++j) {
                    const float4 g = j == back ? h : h_at(t - back + j);
                    fma4(ya, *reinterpret_cast<const float4*>(a.wa + static_cast<uint64_t>(j) * a.ld + c), g);
                    if (a.wb) fma4(yb, *reinterpret_cast<const float4*>(a.wb + static_cast<uint64_t>(j) * a.ld + c), g);
                }
                store(t, ya, yb);
            }
        }
    }
}

template <typename T>
__global__ __launch_bounds__(256) void concat2_kernel(const float* __restrict__ a, const float* __restrict__ b, uint64_t ld, T* __restrict__ out) {
    const uint64_t c = (static_cast<uint64_t>(blockIdx.x) * 256 + threadIdx.x) * 4, t = blockIdx.y;
    if (c >= 2 * ld) return;
    const float4 v = *reinterpret_cast<const float4*>(c < ld ? a + t * ld + c : b + t * ld + (c - ld));
    ElemOps<T>::store4(out + t * 2 * ld + c, v.x, v.y, v.z, v.w);
}

}  // namespace

cera_hip_status cera_launch_embed_pos(cera_hip_ctx* ctx, const void* embed, const void* pos, const uint32_t* tokens, uint32_t token,
                                      uint32_t n, uint32_t start, uint32_t width, uint64_t ld, float* x, float* x0) {
    hipLaunchKernelGGL(embed_pos_kernel, dim3(static_cast<uint32_t>((ld + 255) / 256), n), dim3(256), 0, ctx->stream,
                       static_cast<const uint16_t*>(embed), static_cast<const uint16_t*>(pos), tokens, token, start, width, ld, x, x0);
    HIP_TRY(ctx, hipGetLastError());
    return CERA_HIP_OK;
}

cera_hip_status cera_launch_embed_streams(cera_hip_ctx* ctx, const void* embed, const uint32_t* tokens, uint32_t token, uint32_t n, uint32_t width,
                                          uint64_t ld, float* x, uint32_t streams, uint64_t stride, float u_scale, float* u) {
    if (ld % 4 || stride % 4) return cera_fail(ctx, CERA_HIP_ERR_SHAPE, "embed_streams: rows in whole vectors");
    hipLaunchKernelGGL(embed_streams_kernel, dim3(static_cast<uint32_t>((ld + 1023) / 1024), n), dim3(256), 0, ctx->stream,
                       static_cast<const uint16_t*>(embed), tokens, token, width, ld, x, streams, stride, u_scale, u);
    HIP_TRY(ctx, hipGetLastError());
    return CERA_HIP_OK;
}

cera_hip_status cera_launch_norm_conv(cera_hip_ctx* ctx, const NormConv& a, bool f32) {
    if (a.ld % 4 || a.taps > CONV_MAX_TAPS || (a.taps > 1 && (!a.ring.rows || a.ring.depth < a.taps)) || (a.out_b && !a.wb && a.taps))
        return cera_fail(ctx, CERA_HIP_ERR_SHAPE, "norm_conv: bad shape");
    // one workgroup per CU, more rows each beyond that
    const int rows = static_cast<int>(std::min<uint32_t>(NC_MAX_ROWS, std::max<uint32_t>(1, (a.n + ctx->n_cu - 1) / ctx->n_cu)));
    const dim3 grid((a.n + rows - 1) / rows), block(NC_WAVES * 64);
    auto go = [&](auto tag) {
        using T = decltype(tag);
        switch (a.taps) {
            case 2: hipLaunchKernelGGL((norm_conv_kernel<T, 2>), grid, block, 0, ctx->stream, a, rows); break;
            case 3: hipLaunchKernelGGL((norm_conv_kernel<T, 3>), grid, block, 0, ctx->stream, a, rows); break;
            case 4: hipLaunchKernelGGL((norm_conv_kernel<T, 4>), grid, block, 0, ctx->stream, a, rows); break;
            default: hipLaunchKernelGGL((norm_conv_kernel<T, 0>), grid, block, 0, ctx->stream, a, rows); break;
        }
    };
    if (f32) go(float{});
    else go(static_cast<__bf16>(0.0f));
    HIP_TRY(ctx, hipGetLastError());
    return CERA_HIP_OK;
}

cera_hip_status cera_launch_concat2(cera_hip_ctx* ctx, const float* a, const float* b, uint32_t n, uint64_t ld, void* out, bool f32) {
    const dim3 grid(static_cast<uint32_t>((2 * ld / 4 + 255) / 256), n);
    if (f32) hipLaunchKernelGGL(concat2_kernel<float>, grid, dim3(256), 0, ctx->stream, a, b, ld, static_cast<float*>(out));
    else hipLaunchKernelGGL(concat2_kernel<__bf16>, grid, dim3(256), 0, ctx->stream, a, b, ld, static_cast<__bf16*>(out));
    HIP_TRY(ctx, hipGetLastError());
    return CERA_HIP_OK;
}
