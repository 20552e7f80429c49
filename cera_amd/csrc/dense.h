// Launchers of the float-weight (bfloat16) matrix products: a matrix-core GEMM for many rows of
// activations and a streaming GEMV for one, with the small operations around them folded in.
#pragma once
#include "host_common.h"
#include "sigmoid_attn.h"   // SAttnPartials

constexpr uint32_t DENSE_PAD = 64;   // K is padded with zeros to whole 128-byte lines of bf16
static inline uint64_t dense_pad(uint64_t k) { return (k + DENSE_PAD - 1) / DENSE_PAD * DENSE_PAD; }

// bf16 weights [rows][kp] in HBM.  kp: a multiple of DENSE_PAD, the pad columns zero.
struct DenseMat {
    void* w = nullptr;
    uint32_t rows = 0, kp = 0;
};

// What happens to the products y[row]:
enum DenseEpilogue {
    DENSE_STORE = 0,    // out[row] = y (+ bias[row])                        f32
    DENSE_ADD = 1,      // out[row] += mult * y                              f32
    DENSE_SWIGLU = 2,   // rows come in groups of 16 gate rows then 16 up rows: out[i] = silu(gate_i) * up_i   element type
    DENSE_CAST = 3,     // out[row] = y                                       element type
    DENSE_RELU2 = 4,    // out[row] = max(y, 0)^2                             element type
    DENSE_STREAMS = 5   // adds y to several residual streams at once (DenseStreams)          f32
};
// Residual streams x_0 .. x_{count-1}: x_t <- sum_s mix[s][t] x_s + out[t] y, all from the old ones, and the next
// reader's input u = sum_t next[t] x_t on the way.  DenseOut::out is x_0, the others follow `stride` floats apart.
constexpr uint32_t DENSE_MAX_STREAMS = 8;
struct DenseStreams {
    uint32_t count = 0;
    uint64_t stride = 0;
    float out[DENSE_MAX_STREAMS] = {}, next[DENSE_MAX_STREAMS] = {};
    float mix[DENSE_MAX_STREAMS][DENSE_MAX_STREAMS] = {};   // [from][to]
};
struct DenseOut {
    int epi = DENSE_STORE;
    void* out = nullptr;
    uint64_t ld = 0;              // elements between tokens
    const float* bias = nullptr;  // DENSE_STORE, nullable
    float mult = 1.0f;            // DENSE_ADD
    uint32_t rows = 0;            // output elements per token
    const DenseStreams* streams = nullptr;   // DENSE_STREAMS, host
    float* u = nullptr;                      // DENSE_STREAMS: the next reader's input, rows as x's
};
// Several products of the same shape in one launch, as the heads of a layer have them: number g reads rows
// [g * w.rows / count, ...) of the matrix and its own columns of x, and writes its own columns of out.
struct DenseGroups {
    uint32_t count = 1;
    uint64_t x_stride = 0, out_stride = 0;   // elements between the groups' x and out
};

// many tokens: x [n][ldx] of bf16 (f32 == false) or float, ldx >= w.kp
cera_hip_status cera_launch_dense_gemm(cera_hip_ctx* ctx, const DenseMat& w, const void* x, uint64_t ldx, uint32_t n,
                                       const DenseOut& o, bool f32, const DenseGroups& groups = {});

// One token.  Where its activations come from:
struct DenseIn {
    // RAW: element-type vector [kp].  NORM: x f32 [kp], normalised over its first n_mean entries.
    // MERGE: as RAW, but the first heads * vdim elements are the sum of attention's partial results.
    // CONCAT: x | x2, f32 [kp / 2] each.  Pad columns of x, x2, scale, add and plain are zero.
    enum Kind { RAW = 0, NORM = 1, CONCAT = 2, MERGE = 3 } kind = RAW;
    const void* x = nullptr;
    const float* x2 = nullptr;
    uint32_t n_mean = 0;
    float eps = 0;
    SAttnPartials merge;
    // NORM: staged value of channel c is x[c] * inv * scale[c] + (add ? add[c] : 0)
    const float *scale_a = nullptr, *add_a = nullptr, *scale_b = nullptr, *add_b = nullptr;
    // NORM: also h[c] = x[c] * inv * plain[c] into h_out (nullable), by one workgroup
    const float* plain = nullptr;
    float* h_out = nullptr;
};
// y = W_a . in_a, and in the same launch y_b = W_b . in_b (wb nullable).  The two may have different
// NORM scale / add vectors; the other kinds share the one input.  *launched = false when the input
// does not fit the workgroup's LDS (the caller then takes the GEMM route).
cera_hip_status cera_launch_dense_gemv(cera_hip_ctx* ctx, const DenseIn& in, const DenseMat& wa, const DenseOut& oa,
                                       const DenseMat* wb, const DenseOut* ob, bool f32, bool* launched);
// whether a product with inputs of kp elements has a GEMV
bool cera_dense_gemv_fits(uint64_t kp, bool f32);
