// Causal softmax attention with a sink per head, over a cache of key | value rows.
//
//   weight(i, j) = exp(scale * q_i . k_j) / (exp(sink_h) + sum_{j' <= i} exp(scale * q_i . k_j'))
//
// The cache of one key/value head holds, per position, one row of `row` elements T (bf16 or f32): key columns
// [0, kp) and value columns [v_off, v_off + vp).  The two may overlap: attention over compressed rows uses the
// same columns for both.  Pads are zero and every entry is finite from the start; positions come in whole
// steps of 64.
#pragma once
#include "host_common.h"
#include "sigmoid_attn.h"   // SAttnPartials

constexpr uint32_t FATTN_CAP_STEP = 64;
constexpr uint32_t FATTN_MAX_KEY = 576, FATTN_MAX_VALUE = 512, FATTN_MAX_ROW = 640;   // padded columns
static inline uint32_t fattn_pad(uint32_t d, uint32_t to) { return (d + to - 1) / to * to; }

struct FAttnShape {
    uint32_t heads = 0, kv_heads = 0;
    uint32_t kp = 0;              // key columns, a multiple of 32
    uint32_t v_off = 0, vp = 0;   // first value column (a multiple of 64) and their number (of 32)
    uint32_t vdim = 0;            // value columns that are written out
    uint32_t row = 0;             // elements of a row, a multiple of 64
    float scale = 1.0f;
    const float* sink = nullptr;  // [heads], device
};
// rows of separate keys and values
static inline FAttnShape fattn_shape(uint32_t heads, uint32_t kv_heads, uint32_t dim, uint32_t vdim, float scale, const float* sink) {
    FAttnShape s;
    s.heads = heads; s.kv_heads = kv_heads; s.kp = fattn_pad(dim, 32); s.v_off = fattn_pad(dim, 64); s.vp = fattn_pad(vdim, 32);
    s.vdim = vdim; s.row = fattn_pad(s.v_off + s.vp, 64); s.scale = scale; s.sink = sink;
    return s;
}

// One pass over n tokens from position `start`.
struct FAttnPass {
    uint32_t n = 0, start = 0;
    const void* q = nullptr;      // [n][heads][kp] T
    void* kv = nullptr;           // [kv_heads][cap][row] T
    uint32_t cap = 0;
    void* out = nullptr;          // [n][out_ld] T, head h at column h * out_head
    uint64_t out_ld = 0;
    uint32_t out_head = 0;
};
bool cera_fattn_fits(const FAttnShape& s);
// merge (nullable, n == 1): receives partial results over at most `most` key ranges that the consumer adds up itself --
// or part == nullptr when the launch has already written p.out, as it does beyond that
cera_hip_status cera_launch_fattn(cera_hip_ctx* ctx, const FAttnShape& s, const FAttnPass& p, SAttnPartials* merge, uint32_t most, bool f32);

// What stands between the projections and attention in a layer with separate keys and values: norms over the
// entries of each query and key head, a factor per position on the queries, values mixed with another layer's
// values of the same token, and the append.
struct FAttnPrep {
    const float* qkv = nullptr;       // [n][ld]: q | k | v
    uint64_t ld = 0;
    uint32_t dim = 0;
    const float *q_norm = nullptr, *k_norm = nullptr;   // [dim]
    float eps = 0;
    const float* q_mult = nullptr;    // [position], nullable
    float* v_first = nullptr;         // [n][kv_heads * vdim], nullable
    bool v_store = false;             // v_first receives this layer's values; else they are mixed in
    float v_lambda = 0;               // v <- (1 - lambda) v + lambda v_first
};
// q [n][heads][kp] goes to p.q, keys and values into p.kv
cera_hip_status cera_launch_fattn_prep(cera_hip_ctx* ctx, const FAttnShape& s, const FAttnPass& p, const FAttnPrep& a, bool f32);
