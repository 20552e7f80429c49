// Attention over compressed key/value rows: a token's cache row holds a latent c (normalised) and one rotated key
// part shared by all heads; head h's key is [W_uk,h c | shared part] and its value W_uv,h c.
//
// Two ways to the same numbers.  Absorbed: q_h' = W_uk,h^T q_h meets c itself, attention has one kv head whose rows
// serve as keys and values, and W_uv,h follows.  Expanded: keys and values of every head are written out for the
// positions in reach, then ordinary attention runs over them -- fewer operations per (query, key) pair, once many
// queries share the expansion.
#pragma once
#include "dense.h"
#include "softmax_attn.h"

struct LatentShape {
    uint32_t heads = 0, dim = 0, rot_dim = 0, vdim = 0, rank = 0;
    uint32_t rot_dims = 0;              // leading entries of the rotated part that turn, in adjacent pairs
    const float* rot_table = nullptr;   // [position][rot_dims / 2] (cos, sin), device
    const float* c_norm = nullptr;      // [rank]
    float eps = 0;
    uint32_t rank_p() const { return static_cast<uint32_t>(dense_pad(rank)); }
    uint32_t dim_p() const { return static_cast<uint32_t>(dense_pad(dim)); }
};
// the cache's row and attention over it: c at column 0, the shared key part at column rank_p
static inline FAttnShape latent_absorbed(const LatentShape& l, float scale, const float* sink) {
    FAttnShape s;
    s.heads = l.heads; s.kv_heads = 1; s.kp = l.rank_p() + fattn_pad(l.rot_dim, 32); s.v_off = 0; s.vp = s.vdim = l.rank_p();
    s.row = fattn_pad(s.kp, 64); s.scale = scale; s.sink = sink;
    return s;
}
static inline FAttnShape latent_expanded(const LatentShape& l, float scale, const float* sink) {
    return fattn_shape(l.heads, l.heads, l.dim + l.rot_dim, l.vdim, scale, sink);
}

// Behind the projections x [n][ld] = q | down (q per head: dim unrotated, rot_dim rotated; down: rank, rot_dim):
// appends the rows of positions start .. to `cache` ([cap][row] of the absorbed shape) and lays the queries out.
//   absorbed: unrotated parts to qn [n][heads][dim_p], rotated parts into q [n][heads][kp] from column rank_p on
//   expanded (qn null): both parts side by side in q [n][heads][kp]
cera_hip_status cera_launch_latent_prep(cera_hip_ctx* ctx, const LatentShape& l, const FAttnShape& absorbed, const float* x, uint64_t ld, uint32_t n,
                                        uint32_t start, void* cache, void* q, uint32_t kp, void* qn, bool f32);
// Expanded rows [heads][cap][row]: the shared key part of positions 0 .. total - 1 beside each head's unrotated
// columns, zeros in the pads and in the rows up to the next multiple of 64.
cera_hip_status cera_launch_latent_spread(cera_hip_ctx* ctx, const LatentShape& l, const FAttnShape& absorbed, const FAttnShape& expanded,
                                          const void* cache, uint32_t total, void* rows, uint32_t cap, bool f32);

// One token, absorbed: the preparation above and q' = W_uk^T q in one launch.  wk [heads][rank_p][dim_p].
cera_hip_status cera_launch_latent_step(cera_hip_ctx* ctx, const LatentShape& l, const FAttnShape& absorbed, const DenseMat& wk, const float* x,
                                        uint32_t pos, void* cache, void* q, bool f32);
// One token: adds attention's partial results up (at most LATENT_PARTS; parts.part null: `merged` [heads][rank_p] T holds
// the sum) and applies W_uv; wv [heads * vdim][rank_p], out T, head h at h * vdim.
constexpr uint32_t LATENT_PARTS = 32;
cera_hip_status cera_launch_latent_values(cera_hip_ctx* ctx, const LatentShape& l, const DenseMat& wv, const SAttnPartials& parts, const void* merged,
                                          void* out, bool f32);
