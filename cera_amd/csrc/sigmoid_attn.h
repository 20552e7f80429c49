// Attention with unnormalised sigmoid weights over a chunked causal mask, a gate per head, and its
// KV cache.
//
//   weight(i, j) = sigmoid(scale * q_i . k_j + bias_h)   for j <= i in the same chunk as i, else 0
//   out_h(i)     = gate_h(i) * sum_j weight(i, j) v_j
//
// A chunk is `chunk` consecutive positions counted from position 0 of the sequence (0: no chunks).
//
// Cache of one layer, element type T (bf16 or f32): K [kv_heads][cap][dim_p], V transposed
// [kv_heads][vdim_p][cap].  dim_p and vdim_p are the head sizes rounded up to 32 (pad columns zero),
// cap the positions rounded up to 64; every entry is finite from the start.  With V transposed, both
// matrix products read their cache operand in 16-byte runs and no operand passes through LDS.
#pragma once
#include "host_common.h"

constexpr uint32_t SATTN_CAP_STEP = 64;   // cache positions come in whole steps of this
static inline uint32_t sattn_pad32(uint32_t d) { return (d + 31) / 32 * 32; }

struct SAttnShape {
    uint32_t heads = 0, kv_heads = 0, dim = 0, vdim = 0;
    uint32_t chunk = 0;
    float scale = 1.0f;
    uint32_t rot_dims = 0;
    const float* rot_table = nullptr;   // [position][rot_dims / 2] (cos, sin), device
    const float* bias = nullptr;        // [heads], device
};

// One pass over n tokens from position `start`.
struct SAttnPass {
    const float* qkvg = nullptr;   // [n][ld] projections: q | k | v | gate, unrotated
    uint64_t ld = 0;
    uint32_t n = 0, start = 0;
    void *kc = nullptr, *vc = nullptr;
    uint32_t cap = 0;
    void* q = nullptr;             // [n][heads][dim_p] T: rotated queries (written by the append, read by attention)
    void* out = nullptr;           // [n][out_ld] T, head h at column h * vdim
    uint64_t out_ld = 0;
};

// The rows a layer's input convolutions keep: h of position p in row p % depth.
struct ConvRing {
    float* rows = nullptr;   // [depth][ld]
    uint32_t depth = 0, width = 0;
    uint64_t ld = 0;
};

// K (rotated) and V of the pass into the cache, rotated q into p.q, and -- x given -- the pass's last
// normalised rows x * inv * w into the convolution ring.
cera_hip_status cera_launch_sattn_append(cera_hip_ctx* ctx, const SAttnShape& s, const SAttnPass& p, const ConvRing& ring,
                                         const float* x, uint64_t x_ld, const float* inv, const float* w, bool f32);
cera_hip_status cera_launch_sattn(cera_hip_ctx* ctx, const SAttnShape& s, const SAttnPass& p, bool f32);
// The decode step's form, n == 1: rotation and append inside the attention launch.  Extra workgroups add up
// the convolutions' history for the position after this one (hist_a / hist_b, [width] each) when ring.rows.
struct ConvHist {
    const float *wa = nullptr, *wb = nullptr;   // [taps][width]; wb nullable
    uint32_t taps = 0;
    float *a = nullptr, *b = nullptr;
};
// merge (nullable): receives partial results over key ranges that the consumer of the output adds up and gates
// itself -- or part == nullptr when the launch has already written p.out.
constexpr uint32_t SATTN_MERGE_SPLITS = 8;
constexpr uint32_t PARTIALS_MAX = 2048;   // heads * splits a consumer takes
struct SAttnPartials {
    const float* part = nullptr;   // [splits][heads][vdim_p]
    const float* gate = nullptr;   // sigmoid weights: [heads], before the sigmoid
    // softmax weights: maximum (in powers of two) and sum of every part, [splits][heads][2], and the heads' sinks
    const float *ml = nullptr, *sink = nullptr;
    uint32_t splits = 0, heads = 0, vdim = 0, vdim_p = 0;
};
cera_hip_status cera_launch_sattn_step(cera_hip_ctx* ctx, const SAttnShape& s, const SAttnPass& p, const ConvRing& ring,
                                       const ConvHist& hist, SAttnPartials* merge, bool f32);
// the history sums alone, for the token at `pos`
cera_hip_status cera_launch_conv_hist(cera_hip_ctx* ctx, const ConvRing& ring, const ConvHist& hist, uint32_t pos);
