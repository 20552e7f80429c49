// Row kernels of the layered float models: embedding with learned positions, row norm with the
// input convolutions, concatenation of two residual streams.
#pragma once
#include "host_common.h"
#include "sigmoid_attn.h"   // ConvRing

// x[t] = x0[t] = embed[token[t]] + pos[start + t]; ld floats per row, pad columns written zero.  tokens: device.
cera_hip_status cera_launch_embed_pos(cera_hip_ctx* ctx, const void* embed, const void* pos, const uint32_t* tokens, uint32_t token,
                                      uint32_t n, uint32_t start, uint32_t width, uint64_t ld, float* x, float* x0);

// x_s[t] = embed[token[t]] for every one of `streams` streams, `stride` floats apart, and u[t] = u_scale * embed[token[t]]
cera_hip_status cera_launch_embed_streams(cera_hip_ctx* ctx, const void* embed, const uint32_t* tokens, uint32_t token, uint32_t n, uint32_t width,
                                          uint64_t ld, float* x, uint32_t streams, uint64_t stride, float u_scale, float* u);

// h = rmsnorm(x) per row; out_a = h + conv(h; wa), out_b likewise (nullable), T [n][ld].  wa / wb:
// [taps][ld] f32, tap taps-1 the current position; taps == 0: out_a = h.  Rows before the pass come from the ring.
struct NormConv {
    const float* x = nullptr;
    uint64_t ld = 0;
    uint32_t n = 0, start = 0, width = 0, taps = 0;
    float eps = 0;
    const float *w = nullptr, *wa = nullptr, *wb = nullptr;
    ConvRing ring;
    void *out_a = nullptr, *out_b = nullptr;
    float* inv = nullptr;   // [n] 1 / rms of each row (nullable)
};
constexpr uint32_t CONV_MAX_TAPS = 32;
cera_hip_status cera_launch_norm_conv(cera_hip_ctx* ctx, const NormConv& a, bool f32);

// out[t] = a[t] | b[t], T [n][2 ld]
cera_hip_status cera_launch_concat2(cera_hip_ctx* ctx, const float* a, const float* b, uint32_t n, uint64_t ld, void* out, bool f32);
