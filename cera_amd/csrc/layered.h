// State of the layered float model family (layered.hip: parallel blocks and what both forms share;
// layered_seq.hip: sequential blocks over several residual streams).
#pragma once
#include <map>
#include <tuple>

#include "conv_norm.h"
#include "copy_budget.h"
#include "dense.h"
#include "latent.h"
#include "model.h"
#include "sigmoid_attn.h"
#include "softmax_attn.h"

// ---- parallel blocks ----
struct LayerW {
    SAttnShape shape;
    DenseMat qkvg, gate_up, down;      // down: O | down side by side
    uint32_t ff = 0;
    uint64_t att_p = 0;                // columns of the attention output in down's input
    float *norm = nullptr, *conv_a = nullptr, *conv_b = nullptr;    // [ld], [taps][ld]
    float *scale_a = nullptr, *scale_b = nullptr;                   // norm * (1 + last tap)
};
// One pass over a layer, with its own cache and state
struct Run {
    uint32_t layer = 0;
    int step = -1;                     // number of the pass that begins here, or -1
    void *kc = nullptr, *vc = nullptr;
    ConvRing ring;
    ConvHist hist;
};

// ---- sequential blocks ----
struct SeqLayer {
    bool latent = false;
    uint32_t dim = 0, vdim = 0, kv_heads = 0, ff = 0;
    FAttnShape attn, wide;             // the cache's rows; latent: the expanded rows
    LatentShape lat;
    FAttnPrep prep;                    // softmax mixer: what does not change between passes
    bool v_mix = false;
    DenseMat in;                       // q | k | v, or q | kv_down
    DenseMat k_up, k_up_t, v_up;       // latent: [heads * dim][rank_p], [heads][rank_p][dim_p], [heads * vdim][rank_p]
    DenseMat o, up, down;
    float *norm = nullptr, *norm_ffn = nullptr;
    DenseStreams st_mixer, st_ffn;     // stride 0: set per pass
    void* kv = nullptr;                // cache
};

struct CeraLayered {
    cera_hip_layered_config cfg{};
    bool f32 = false;
    uint32_t esz = 2;                  // bytes of an activation / cache element
    uint64_t ld = 0;                   // floats of a residual row: width padded
    uint32_t cap = 0;                  // cache positions
    uint32_t steps = 0;                // rows of loop_step
    std::vector<LayerW> layers;
    std::vector<Run> runs;
    std::vector<SeqLayer> seq;
    void *embed = nullptr, *pos = nullptr;
    DenseMat head, loop_in;
    float *loop_step = nullptr, *final_norm = nullptr;
    bool step_fits = true;             // every decode product's input fits the GEMV's LDS
    // one token
    float *x = nullptr, *xb = nullptr, *x0 = nullptr, *qkvg = nullptr;
    void *cat = nullptr, *q = nullptr;
    // state of the sequence
    uint32_t hist_pos = UINT32_MAX;    // position the convolution history sums are for
    uint32_t ring_lo = 0;              // oldest position the rings still hold
    // batched pass, token-major, `cap_n` rows
    uint32_t cap_n = 0;
    float *bx = nullptr, *bx0 = nullptr, *bqkvg = nullptr, *binv = nullptr;
    void *ba = nullptr, *bb = nullptr, *bq = nullptr, *bcat = nullptr, *bcat2 = nullptr;
    uint32_t* btok = nullptr;
    float* blogits = nullptr;
    uint32_t logits_cap = 0;
    uint64_t b_bytes = 0;
    std::vector<void*> b_owned;
    // sequential blocks: x holds all streams; the next sublayer's input, feed-forward activations, first mixing layer's values
    float u_scale = 1.0f;              // what the first sublayer reads of the embedding
    float *u = nullptr, *v_first = nullptr, *bu = nullptr, *bv_first = nullptr;
    void *act = nullptr, *lat = nullptr, *bqn = nullptr, *bo = nullptr;
};

// ---- shared between the two forms (layered.hip) ----
cera_hip_status layered_alloc(cera_hip_model* m, uint64_t bytes, void** out, bool zero);
template <class T> cera_hip_status layered_alloc_t(cera_hip_model* m, uint64_t n, T** out, bool zero = true) {
    return layered_alloc(m, n * sizeof(T), reinterpret_cast<void**>(out), zero);
}
// a host vector of n floats into ld floats (pad zero)
cera_hip_status layered_put_vec(cera_hip_model* m, const float* src, uint64_t n, uint64_t ld, float** out);
// pass buffers, freed together when a longer pass comes
cera_hip_status layered_batch_alloc(cera_hip_model* m, uint64_t bytes, void** out);
void layered_batch_free(cera_hip_model* m);
cera_hip_status layered_batch_logits(cera_hip_model* m, uint32_t n);
// rotation tables by their constants
typedef std::map<std::tuple<uint32_t, double, uint32_t, double, double, double, double>, float*> RotationTables;
cera_hip_status layered_rotation(cera_hip_model* m, const cera_hip_attn_spec& s, RotationTables* tables, const float** out);
// bf16 rows of several matrices packed into one padded matrix
struct Packer {
    std::vector<uint16_t> host;
    uint64_t kp = 0;
    Packer(uint64_t rows, uint64_t kp_) : host(rows * kp_, 0), kp(kp_) {}
    void row(uint64_t dst, uint64_t col, const cera_hip_tensor& t, uint64_t src, uint64_t c0 = 0, uint64_t n = 0);
    void rows(uint64_t dst, uint64_t col, const cera_hip_tensor& t);
    cera_hip_status put(cera_hip_model* m, DenseMat* out);
};
// a cached element <-> float, rounding as the kernels do
float layered_get(const CeraLayered& g, const void* rows, uint64_t i);
void layered_set(const CeraLayered& g, void* rows, uint64_t i, float f);

// ---- sequential blocks (layered_seq.hip) ----
const CeraModelOps* layered_seq_ops();
cera_hip_status layered_seq_check(cera_hip_ctx* ctx, const cera_hip_layered_config& c, const cera_hip_layered_layer* layers);
cera_hip_status layered_seq_build(cera_hip_model* m, const cera_hip_layered_config& c, const cera_hip_layered_layer* layers);
void layered_destroy(cera_hip_model* m);
// n tokens from start_pos on through `pass`, in portions of one pass
typedef cera_hip_status (*LayeredPass)(cera_hip_model* m, const uint32_t* tokens, uint32_t n, uint32_t start, bool last, float* all);
cera_hip_status layered_portions(cera_hip_model* m, LayeredPass pass, const uint32_t* tokens, uint32_t n, uint32_t start, float* last_logits, float* all);
// shape and type of a caller's matrix
cera_hip_status layered_mat(cera_hip_ctx* ctx, const cera_hip_tensor& t, uint64_t m, uint64_t k, const char* name);
cera_hip_status layered_bad(cera_hip_ctx* ctx, const std::string& what);
