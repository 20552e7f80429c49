// Sequential blocks of the layered float family: mixer, then feed-forward, each behind its own norm, over several
// residual streams.
//
// Writing to the streams and reading the next sublayer's input from them are both channel by channel, so one
// epilogue does both: the output product of a sublayer updates all streams and leaves u = sum_t next[t] x_t, and
// every norm reads a single row however many streams there are.
//
// Decode, per layer: [norm, projections] - [norms, query factor, value mixing, append] - [attention] - [O, which adds up
// attention's partial results; streams] - [norm, up, relu^2] - [down; streams].  A latent mixer has [append and
// absorbed queries] - [attention] - [sum of the partial results, values] in the middle.
#include <algorithm>
#include <cmath>
#include <cstring>

#include "layered.h"

namespace {

using L = CeraLayered;

// expanded rows of a latent mixer beyond this stay compressed
constexpr uint64_t EXPAND_MAX_BYTES = 2ull << 30;

DenseOut to_streams(const DenseStreams& st, float* x, float* u, uint64_t ld, uint32_t width) {
    DenseOut o;
    o.epi = DENSE_STREAMS; o.out = x; o.u = u; o.ld = ld; o.rows = width; o.streams = &st;
    return o;
}

cera_hip_status seq_pass(cera_hip_model* m, const uint32_t* tokens, uint32_t n, uint32_t start, bool last, float* all);

// logits of the row u through the final norm
cera_hip_status row_logits(cera_hip_model* m, const float* u) {
    L& g = *m->layered;
    DenseIn in;
    in.kind = DenseIn::NORM; in.x = u; in.n_mean = g.cfg.width; in.eps = g.cfg.eps; in.scale_a = g.final_norm;
    DenseOut out;
    out.out = m->logits; out.rows = g.cfg.vocab;
    bool ok = false;
    CERA_TRY(cera_launch_dense_gemv(m->ctx, in, g.head, out, nullptr, nullptr, g.f32, &ok));
    return ok ? CERA_HIP_OK : cera_fail(m->ctx, CERA_HIP_ERR_SHAPE, "logits: the row does not fit the GEMV");
}

// ---- the decode step ------------------------------------------------------------------------------
cera_hip_status seq_decode(cera_hip_model* m, uint32_t token, uint32_t pos, bool want_logits) {
    L& g = *m->layered;
    cera_hip_ctx* ctx = m->ctx;
    if (!g.step_fits) return seq_pass(m, &token, 1, pos, want_logits, nullptr);
    const uint32_t width = g.cfg.width;
    auto gemv = [&](const DenseIn& in, const DenseMat& w, const DenseOut& out) {
        bool ok = false;
        cera_hip_status st = cera_launch_dense_gemv(ctx, in, w, out, nullptr, nullptr, g.f32, &ok);
        if (st == CERA_HIP_OK && !ok) st = cera_fail(ctx, CERA_HIP_ERR_SHAPE, "decode: a product's input does not fit the GEMV");
        return st;
    };
    auto streams = [&](DenseStreams& st) {
        st.stride = g.ld;
        return to_streams(st, g.x, g.u, g.ld, width);
    };
    CERA_TRY(cera_launch_embed_streams(ctx, g.embed, nullptr, token, 1, width, g.ld, g.x, g.cfg.streams, g.ld, g.u_scale, g.u));
    for (SeqLayer& W : g.seq) {
        DenseIn in;
        in.kind = DenseIn::NORM; in.x = g.u; in.n_mean = width; in.eps = g.cfg.eps; in.scale_a = W.norm;
        DenseOut proj;
        proj.out = g.qkvg; proj.rows = W.in.rows;
        CERA_TRY(gemv(in, W.in, proj));
        FAttnPass p;
        p.n = 1; p.start = pos; p.kv = W.kv; p.cap = g.cap; p.q = g.q;
        DenseIn raw;
        raw.x = g.cat;
        if (W.latent) {
            CERA_TRY(cera_launch_latent_step(ctx, W.lat, W.attn, W.k_up_t, g.qkvg, pos, W.kv, g.q, g.f32));
            SAttnPartials parts;
            p.out = g.lat; p.out_head = W.lat.rank_p(); p.out_ld = 0;
            CERA_TRY(cera_launch_fattn(ctx, W.attn, p, &parts, LATENT_PARTS, g.f32));
            CERA_TRY(cera_launch_latent_values(ctx, W.lat, W.v_up, parts, g.lat, g.cat, g.f32));
        } else {
            FAttnPrep prep = W.prep;
            prep.qkv = g.qkvg; prep.ld = W.in.rows; prep.v_first = W.v_mix ? g.v_first : nullptr;
            CERA_TRY(cera_launch_fattn_prep(ctx, W.attn, p, prep, g.f32));
            p.out = g.cat; p.out_head = W.vdim; p.out_ld = W.o.kp;
            // every workgroup of the output product reads all parts: 64 KB of them at the most
            const uint32_t most = std::min(8u, std::max(1u, 16384u / (W.attn.heads * W.attn.vp)));
            CERA_TRY(cera_launch_fattn(ctx, W.attn, p, &raw.merge, most, g.f32));
            if (raw.merge.part) raw.kind = DenseIn::MERGE;
        }
        CERA_TRY(gemv(raw, W.o, streams(W.st_mixer)));
        if (!W.ff) continue;
        in.scale_a = W.norm_ffn;
        DenseOut act;
        act.epi = DENSE_RELU2; act.out = g.act; act.rows = W.ff;
        CERA_TRY(gemv(in, W.up, act));
        DenseIn down;
        down.x = g.act;
        CERA_TRY(gemv(down, W.down, streams(W.st_ffn)));
    }
    m->hidden = g.u;
    return want_logits ? row_logits(m, g.u) : CERA_HIP_OK;
}

// ---- the batched pass -----------------------------------------------------------------------------
cera_hip_status ensure_batch(cera_hip_model* m, uint32_t n, bool logits) {
    L& g = *m->layered;
    if (g.cap_n < n) {
        HIP_TRY(m->ctx, hipStreamSynchronize(m->ctx->stream));
        layered_batch_free(m);
        const uint64_t N = std::min<uint64_t>(std::min<uint32_t>(CERA_PREFILL_CHUNK, g.cfg.max_seq_len), (n + 255) / 256 * 256);
        uint64_t proj = 0, att = 0, q = 0, qn = 0, lat = 0, ff = 0, first = 0;
        for (const SeqLayer& W : g.seq) {
            proj = std::max<uint64_t>(proj, dense_pad(W.in.rows));
            att = std::max<uint64_t>(att, W.o.kp);
            ff = std::max<uint64_t>(ff, W.down.kp);
            q = std::max<uint64_t>(q, static_cast<uint64_t>(W.attn.heads) * std::max(W.attn.kp, W.wide.kp));
            if (W.latent) {
                qn = std::max<uint64_t>(qn, static_cast<uint64_t>(W.attn.heads) * W.lat.dim_p());
                lat = std::max<uint64_t>(lat, static_cast<uint64_t>(W.attn.heads) * W.attn.vp);
            }
            if (W.v_mix) first = static_cast<uint64_t>(W.kv_heads) * W.vdim;
        }
        auto get = [&]() -> cera_hip_status {
            auto el = [&](uint64_t n_el, void** p) { return n_el ? layered_batch_alloc(m, n_el * g.esz, p) : CERA_HIP_OK; };
            auto fl = [&](uint64_t n_el, float** p) { return n_el ? layered_batch_alloc(m, n_el * 4, reinterpret_cast<void**>(p)) : CERA_HIP_OK; };
            CERA_TRY(fl(N * g.ld * g.cfg.streams, &g.bx));
            CERA_TRY(fl(N * g.ld, &g.bu));
            CERA_TRY(fl(N * proj, &g.bqkvg));
            CERA_TRY(fl(N * first, &g.bv_first));
            CERA_TRY(el(N * g.ld, &g.ba));
            CERA_TRY(el(N * ff, &g.bb));
            CERA_TRY(el(N * att, &g.bcat));
            CERA_TRY(el(N * q, &g.bq));
            CERA_TRY(el(N * qn, &g.bqn));
            CERA_TRY(el(N * lat, &g.bo));
            return layered_batch_alloc(m, N * 4, reinterpret_cast<void**>(&g.btok));
        };
        const cera_hip_status st = get();
        if (st != CERA_HIP_OK) { layered_batch_free(m); return st; }
        g.cap_n = static_cast<uint32_t>(N);
    }
    return logits ? layered_batch_logits(m, n) : CERA_HIP_OK;
}

// Whether n queries from `start` on are cheaper over expanded rows: products per (query, key) pair, the second one
// counted twice as its weights come in two parts, against the expansion's own products, which run at about three
// times the rate.
bool expand_pays(const L& g, const SeqLayer& W, uint32_t n, uint32_t start) {
    const double total = static_cast<double>(start) + n, pairs = n * (start + n / 2.0), up = static_cast<double>(W.lat.rank_p()) * (W.dim + W.vdim) / 3.0;
    if (n < 16 || static_cast<double>(W.wide.heads) * fattn_pad(start + n, FATTN_CAP_STEP) * W.wide.row * g.esz > EXPAND_MAX_BYTES) return false;
    return pairs * (W.wide.kp + 2.0 * W.wide.vp) + total * up < pairs * (W.attn.kp + 2.0 * W.attn.vp) + n * up;
}

cera_hip_status latent_pass(cera_hip_model* m, SeqLayer& W, FAttnPass p) {
    L& g = *m->layered;
    cera_hip_ctx* ctx = m->ctx;
    const LatentShape& l = W.lat;
    const uint64_t ld = dense_pad(W.in.rows);
    DenseGroups heads;
    heads.count = l.heads;
    DenseOut to;
    to.epi = DENSE_CAST;
    if (expand_pays(g, W, p.n, p.start)) {
        const uint32_t total = p.start + p.n, cap = fattn_pad(total, FATTN_CAP_STEP);
        void* rows;
        CERA_TRY(cera_scratch(ctx, 14, static_cast<uint64_t>(l.heads) * cap * W.wide.row * g.esz, &rows));
        CERA_TRY(cera_launch_latent_prep(ctx, l, W.attn, g.bqkvg, ld, p.n, p.start, W.kv, g.bq, W.wide.kp, nullptr, g.f32));
        heads.out_stride = static_cast<uint64_t>(cap) * W.wide.row;
        to.ld = W.wide.row;
        to.out = rows; to.rows = l.dim;
        CERA_TRY(cera_launch_dense_gemm(ctx, W.k_up, W.kv, W.attn.row, total, to, g.f32, heads));
        to.out = static_cast<char*>(rows) + static_cast<uint64_t>(W.wide.v_off) * g.esz; to.rows = l.vdim;
        CERA_TRY(cera_launch_dense_gemm(ctx, W.v_up, W.kv, W.attn.row, total, to, g.f32, heads));
        CERA_TRY(cera_launch_latent_spread(ctx, l, W.attn, W.wide, W.kv, total, rows, cap, g.f32));
        p.kv = rows; p.cap = cap;
        return cera_launch_fattn(ctx, W.wide, p, nullptr, 0, g.f32);
    }
    CERA_TRY(cera_launch_latent_prep(ctx, l, W.attn, g.bqkvg, ld, p.n, p.start, W.kv, g.bq, W.attn.kp, g.bqn, g.f32));
    heads.x_stride = l.dim_p(); heads.out_stride = W.attn.kp;
    to.out = g.bq; to.ld = static_cast<uint64_t>(l.heads) * W.attn.kp; to.rows = l.rank_p();
    CERA_TRY(cera_launch_dense_gemm(ctx, W.k_up_t, g.bqn, static_cast<uint64_t>(l.heads) * l.dim_p(), p.n, to, g.f32, heads));
    const FAttnPass direct = p;
    p.out = g.bo; p.out_head = l.rank_p(); p.out_ld = static_cast<uint64_t>(l.heads) * l.rank_p();
    CERA_TRY(cera_launch_fattn(ctx, W.attn, p, nullptr, 0, g.f32));
    heads.x_stride = l.rank_p(); heads.out_stride = l.vdim;
    to.out = direct.out; to.ld = direct.out_ld; to.rows = l.vdim;
    return cera_launch_dense_gemm(ctx, W.v_up, g.bo, p.out_ld, p.n, to, g.f32, heads);
}

cera_hip_status seq_pass(cera_hip_model* m, const uint32_t* tokens, uint32_t n, uint32_t start, bool last, float* all) {
    L& g = *m->layered;
    cera_hip_ctx* ctx = m->ctx;
    const uint32_t width = g.cfg.width;
    CERA_TRY(ensure_batch(m, n, all != nullptr));
    CERA_TRY(cera_hip_upload(ctx, g.btok, tokens, n * 4ull));
    const uint64_t stride = g.cap_n * g.ld;
    CERA_TRY(cera_launch_embed_streams(ctx, g.embed, g.btok, 0, n, width, g.ld, g.bx, g.cfg.streams, stride, g.u_scale, g.bu));
    auto norm = [&](const float* x, uint32_t rows, const float* w) {
        NormConv nc;
        nc.x = x; nc.ld = g.ld; nc.n = rows; nc.width = width; nc.eps = g.cfg.eps; nc.w = w; nc.out_a = g.ba;
        return cera_launch_norm_conv(ctx, nc, g.f32);
    };
    auto streams = [&](DenseStreams& st) {
        st.stride = stride;
        return to_streams(st, g.bx, g.bu, g.ld, width);
    };
    for (SeqLayer& W : g.seq) {
        CERA_TRY(norm(g.bu, n, W.norm));
        DenseOut proj;
        proj.out = g.bqkvg; proj.ld = dense_pad(W.in.rows); proj.rows = W.in.rows;
        CERA_TRY(cera_launch_dense_gemm(ctx, W.in, g.ba, g.ld, n, proj, g.f32));
        FAttnPass p;
        p.n = n; p.start = start; p.kv = W.kv; p.cap = g.cap; p.q = g.bq;
        p.out = g.bcat; p.out_ld = W.o.kp; p.out_head = W.vdim;
        if (W.latent) {
            CERA_TRY(latent_pass(m, W, p));
        } else {
            FAttnPrep prep = W.prep;
            prep.qkv = g.bqkvg; prep.ld = proj.ld; prep.v_first = W.v_mix ? g.bv_first : nullptr;
            CERA_TRY(cera_launch_fattn_prep(ctx, W.attn, p, prep, g.f32));
            CERA_TRY(cera_launch_fattn(ctx, W.attn, p, nullptr, 0, g.f32));
        }
        CERA_TRY(cera_launch_dense_gemm(ctx, W.o, g.bcat, W.o.kp, n, streams(W.st_mixer), g.f32));
        if (!W.ff) continue;
        CERA_TRY(norm(g.bu, n, W.norm_ffn));
        DenseOut act;
        act.epi = DENSE_RELU2; act.out = g.bb; act.ld = W.down.kp; act.rows = W.ff;
        CERA_TRY(cera_launch_dense_gemm(ctx, W.up, g.ba, g.ld, n, act, g.f32));
        CERA_TRY(cera_launch_dense_gemm(ctx, W.down, g.bb, W.down.kp, n, streams(W.st_ffn), g.f32));
    }
    m->hidden = g.bu + static_cast<uint64_t>(n - 1) * g.ld;
    if (!last && !all) return CERA_HIP_OK;
    if (!all && cera_dense_gemv_fits(g.ld, g.f32)) return row_logits(m, m->hidden);
    const uint32_t rows = all ? n : 1;
    CERA_TRY(norm(all ? g.bu : m->hidden, rows, g.final_norm));
    DenseOut out;
    out.out = all ? g.blogits : m->logits; out.ld = g.cfg.vocab; out.rows = g.cfg.vocab;
    CERA_TRY(cera_launch_dense_gemm(ctx, g.head, g.ba, g.ld, rows, out, g.f32));
    return all ? cera_hip_download(ctx, all, g.blogits, static_cast<uint64_t>(n) * g.cfg.vocab * 4) : CERA_HIP_OK;
}

cera_hip_status prefill(cera_hip_model* m, const uint32_t* tokens, uint32_t n, uint32_t start, float* last_logits) {
    return layered_portions(m, seq_pass, tokens, n, start, last_logits, nullptr);
}
cera_hip_status prefill_all(cera_hip_model* m, const uint32_t* tokens, uint32_t n, uint32_t start, float* logits) {
    return layered_portions(m, seq_pass, tokens, n, start, nullptr, logits);
}

// ---- state: cache rows <-> time-major f32 [n][kv_heads * dim] / [n][kv_heads * vdim]; latent: [n][rank] / [n][rot_dim] ----
cera_hip_status move_rows(cera_hip_model* m, uint32_t layer, float* k, float* v, uint32_t n, bool read) {
    L& g = *m->layered;
    const SeqLayer& W = g.seq[layer];
    const uint32_t heads = W.attn.kv_heads, row = W.attn.row;
    const uint32_t kd = W.latent ? W.lat.rank : W.dim, vd = W.latent ? W.lat.rot_dim : W.vdim, vo = W.latent ? W.lat.rank_p() : W.attn.v_off;
    std::vector<char> rows;
    for (uint32_t h = 0; h < heads && n; ++h) {
        char* const dev = static_cast<char*>(W.kv) + static_cast<uint64_t>(h) * g.cap * row * g.esz;
        rows.assign(static_cast<uint64_t>(n) * row * g.esz, 0);
        if (read) CERA_TRY(cera_hip_download(m->ctx, rows.data(), dev, rows.size()));
        for (uint64_t t = 0; t < n; ++t) {
            float* const kt = k + (t * heads + h) * kd;
            float* const vt = v + (t * heads + h) * vd;
            for (uint32_t c = 0; c < kd; ++c) {
                if (read) kt[c] = layered_get(g, rows.data(), t * row + c);
                else layered_set(g, rows.data(), t * row + c, kt[c]);
            }
            for (uint32_t c = 0; c < vd; ++c) {
                if (read) vt[c] = layered_get(g, rows.data(), t * row + vo + c);
                else layered_set(g, rows.data(), t * row + vo + c, vt[c]);
            }
        }
        if (!read) CERA_TRY(cera_hip_upload(m->ctx, dev, rows.data(), rows.size()));
    }
    return CERA_HIP_OK;
}
cera_hip_status read_kv(cera_hip_model* m, uint32_t layer, float* k, float* v) { return move_rows(m, layer, k, v, m->seq_len, true); }
cera_hip_status write_kv(cera_hip_model* m, uint32_t layer, const float* k, const float* v, uint32_t n) {
    return move_rows(m, layer, const_cast<float*>(k), const_cast<float*>(v), n, false);
}

// ---- construction ---------------------------------------------------------------------------------
LatentShape latent_shape(const cera_hip_attn_spec& a, float eps) {
    LatentShape l;
    l.heads = a.heads; l.dim = a.dim; l.rot_dim = a.rot_dim; l.vdim = a.vdim; l.rank = a.kv_rank; l.rot_dims = a.rot_dims; l.eps = eps;
    return l;
}

DenseStreams streams_of(const float* p, uint32_t n) {   // in | out | mix
    DenseStreams s;
    s.count = n;
    for (uint32_t t = 0; t < n; ++t) {
        s.out[t] = p[n + t];
        for (uint32_t f = 0; f < n; ++f) s.mix[f][t] = p[2 * n + f * n + t];
    }
    return s;
}

const CeraModelOps OPS = {seq_decode, prefill, prefill_all, nullptr, read_kv, write_kv, nullptr, nullptr, layered_destroy};

}  // namespace

const CeraModelOps* layered_seq_ops() { return &OPS; }

cera_hip_status layered_seq_check(cera_hip_ctx* ctx, const cera_hip_layered_config& c, const cera_hip_layered_layer* layers) {
    auto bad = [&](const std::string& what) { return layered_bad(ctx, what); };
    auto missing = [&](uint32_t i, const char* what) {
        return cera_fail(ctx, CERA_HIP_ERR_ARGUMENT, "layered_create: layer " + std::to_string(i) + ": " + what + " missing");
    };
    auto mat = [&](const cera_hip_tensor& t, uint64_t rows, uint64_t k, const char* name) { return layered_mat(ctx, t, rows, k, name); };
    if (!c.n_layers || !c.width || !c.vocab || !c.max_seq_len) return bad("zero dimension in config");
    if (c.conv_taps || c.loop_times) return bad("sequential blocks have no input convolutions and no loop");
    if (!c.streams || c.streams > CERA_HIP_MAX_STREAMS) return bad("streams must be 1 to " + std::to_string(CERA_HIP_MAX_STREAMS));
    if (!c.final_norm) return cera_fail(ctx, CERA_HIP_ERR_ARGUMENT, "layered_create: final_norm missing");
    CERA_TRY(mat(c.embed, c.vocab, c.width, "embed"));
    CERA_TRY(mat(c.head, c.vocab, c.width, "head"));
    const cera_hip_attn_spec* first = nullptr;   // of the layers whose values mix
    for (uint32_t i = 0; i < c.n_layers; ++i) {
        const cera_hip_layered_layer& Y = layers[i];
        const cera_hip_attn_spec& a = Y.attn;
        const std::string at = "layer " + std::to_string(i) + ": ";
        if (!Y.norm) return missing(i, "norm");
        if (!Y.sink) return missing(i, "sink");
        if (!Y.streams_attn || (Y.ff && !Y.streams_ffn)) return missing(i, "streams");
        if (!a.heads || !a.dim || !a.vdim) return bad(at + "zero dimension");
        const uint64_t H = a.heads, G = a.kv_heads;
        if (a.kind == CERA_HIP_MIXER_SOFTMAX) {
            if (!G || H % G) return bad(at + "heads must be a multiple of kv_heads");
            if (a.rot_dims) return bad(at + "the softmax mixer does not rotate");
            if (!Y.q_norm || !Y.k_norm) return missing(i, "q_norm / k_norm");
            if (a.q_temp_every < 0) return bad(at + "q_temp_every must not be negative");
            if (a.dim > FATTN_MAX_ROW || a.vdim > FATTN_MAX_ROW || !cera_fattn_fits(fattn_shape(a.heads, a.kv_heads, a.dim, a.vdim, 1.0f, nullptr)))
                return bad(at + "head sizes beyond " + std::to_string(FATTN_MAX_ROW) + " key and value entries together");
            if (a.v_mix) {
                if (first && (first->kv_heads != a.kv_heads || first->vdim != a.vdim)) return bad(at + "values of another shape than those they mix with");
                if (!first) first = &a;
            }
            CERA_TRY(mat(Y.q, H * a.dim, c.width, "q"));
            CERA_TRY(mat(Y.k, G * a.dim, c.width, "k"));
            CERA_TRY(mat(Y.v, G * a.vdim, c.width, "v"));
        } else if (a.kind == CERA_HIP_MIXER_LATENT) {
            if (!a.kv_rank || !a.rot_dim || a.rot_dims % 2 || a.rot_dims > a.rot_dim) return bad(at + "kv_rank, rot_dim and an even rot_dims of at most rot_dim");
            const LatentShape l = latent_shape(a, c.eps);
            if (a.dim > FATTN_MAX_ROW || a.vdim > FATTN_MAX_ROW || a.rot_dim > FATTN_MAX_ROW || a.kv_rank > FATTN_MAX_ROW ||
                !cera_fattn_fits(latent_absorbed(l, 1.0f, nullptr)) || !cera_fattn_fits(latent_expanded(l, 1.0f, nullptr)))
                return bad(at + "kv_rank and rot_dim, or head sizes, beyond the attention kernels' limits");
            if (!Y.latent_norm) return missing(i, "latent_norm");
            CERA_TRY(mat(Y.q, H * (a.dim + a.rot_dim), c.width, "q"));
            CERA_TRY(mat(Y.kv_down, a.kv_rank + a.rot_dim, c.width, "kv_down"));
            CERA_TRY(mat(Y.k_up, H * a.dim, a.kv_rank, "k_up"));
            CERA_TRY(mat(Y.v_up, H * a.vdim, a.kv_rank, "v_up"));
        } else {
            return bad(at + "sequential blocks take the softmax and the latent mixer");
        }
        CERA_TRY(mat(Y.o, c.width, H * a.vdim, "o"));
        if (Y.ff) {
            if (!Y.norm_ffn) return missing(i, "norm_ffn");
            CERA_TRY(mat(Y.ffn_up, Y.ff, c.width, "ffn_up"));
            CERA_TRY(mat(Y.ffn_down, c.width, Y.ff, "ffn_down"));
        }
    }
    return CERA_HIP_OK;
}

cera_hip_status layered_seq_build(cera_hip_model* m, const cera_hip_layered_config& c, const cera_hip_layered_layer* layers) {
    L& g = *m->layered;
    const uint64_t ld = g.ld;
    const uint32_t S = c.streams;
    RotationTables tables;
    std::map<std::pair<double, double>, float*> temps;   // factors per position, by their constants
    uint64_t proj = 0, att = 0, q = 0, ff = 0, first = 0, lat = 0, widest = ld;
    auto pack = [&](const cera_hip_tensor& t, DenseMat* out) {
        Packer p(t.m, dense_pad(t.k));
        p.rows(0, 0, t);
        return p.put(m, out);
    };
    g.seq.resize(c.n_layers);
    DenseStreams* before = nullptr;   // the sublayer whose epilogue prepares the next one's input
    auto reads = [&](const float* in) {
        if (before) std::copy(in, in + S, before->next);
        else { g.u_scale = 0.0f; for (uint32_t s = 0; s < S; ++s) g.u_scale += in[s]; }
    };
    for (uint32_t i = 0; i < c.n_layers; ++i) {
        const cera_hip_layered_layer& Y = layers[i];
        const cera_hip_attn_spec& a = Y.attn;
        SeqLayer& W = g.seq[i];
        float* sink;
        CERA_TRY(layered_put_vec(m, Y.sink, a.heads, a.heads, &sink));
        W.dim = a.dim; W.vdim = a.vdim; W.kv_heads = a.kv_heads; W.ff = Y.ff;
        if (a.kind == CERA_HIP_MIXER_LATENT) {
            W.latent = true;
            W.lat = latent_shape(a, c.eps);
            CERA_TRY(layered_rotation(m, a, &tables, &W.lat.rot_table));
            float* cn;
            CERA_TRY(layered_put_vec(m, Y.latent_norm, a.kv_rank, a.kv_rank, &cn));
            W.lat.c_norm = cn;
            W.attn = latent_absorbed(W.lat, a.scale, sink);
            W.wide = latent_expanded(W.lat, a.scale, sink);
            Packer p(Y.q.m + Y.kv_down.m, ld);
            p.rows(0, 0, Y.q);
            p.rows(Y.q.m, 0, Y.kv_down);
            CERA_TRY(p.put(m, &W.in));
            CERA_TRY(pack(Y.k_up, &W.k_up));
            CERA_TRY(pack(Y.v_up, &W.v_up));
            const uint32_t rank_p = W.lat.rank_p();
            Packer t(static_cast<uint64_t>(a.heads) * rank_p, W.lat.dim_p());   // each head's matrix the other way round
            const uint16_t* const src = static_cast<const uint16_t*>(Y.k_up.data);
            for (uint32_t h = 0; h < a.heads; ++h)
                for (uint32_t d = 0; d < a.dim; ++d)
                    for (uint32_t r = 0; r < a.kv_rank; ++r)
                        t.host[(static_cast<uint64_t>(h) * rank_p + r) * t.kp + d] = src[(static_cast<uint64_t>(h) * a.dim + d) * a.kv_rank + r];
            CERA_TRY(t.put(m, &W.k_up_t));
        } else {
            W.attn = fattn_shape(a.heads, a.kv_heads, a.dim, a.vdim, a.scale, sink);
            Packer p(Y.q.m + Y.k.m + Y.v.m, ld);
            p.rows(0, 0, Y.q);
            p.rows(Y.q.m, 0, Y.k);
            p.rows(Y.q.m + Y.k.m, 0, Y.v);
            CERA_TRY(p.put(m, &W.in));
            W.prep.dim = a.dim; W.prep.eps = c.eps;
            float *qn, *kn;
            CERA_TRY(layered_put_vec(m, Y.q_norm, a.dim, a.dim, &qn));
            CERA_TRY(layered_put_vec(m, Y.k_norm, a.dim, a.dim, &kn));
            W.prep.q_norm = qn; W.prep.k_norm = kn;
            if (a.q_temp_every > 0) {
                float*& t = temps[{a.q_temp_coef, a.q_temp_every}];
                if (!t) {
                    std::vector<float> f(g.cap);
                    for (uint32_t pos = 0; pos < g.cap; ++pos) f[pos] = static_cast<float>(1.0 + a.q_temp_coef * std::log(std::floor((pos + 1.0) / a.q_temp_every) + 1.0));
                    CERA_TRY(layered_put_vec(m, f.data(), f.size(), f.size(), &t));
                }
                W.prep.q_mult = t;
            }
            W.v_mix = a.v_mix != 0;
            W.prep.v_store = W.v_mix && !first;
            W.prep.v_lambda = Y.v_mix_lambda;
            if (W.v_mix) first = static_cast<uint64_t>(a.kv_heads) * a.vdim;
        }
        CERA_TRY(pack(Y.o, &W.o));
        CERA_TRY(layered_put_vec(m, Y.norm, c.width, ld, &W.norm));
        reads(Y.streams_attn);
        W.st_mixer = streams_of(Y.streams_attn, S);
        before = &W.st_mixer;
        if (Y.ff) {
            CERA_TRY(pack(Y.ffn_up, &W.up));
            CERA_TRY(pack(Y.ffn_down, &W.down));
            CERA_TRY(layered_put_vec(m, Y.norm_ffn, c.width, ld, &W.norm_ffn));
            reads(Y.streams_ffn);
            W.st_ffn = streams_of(Y.streams_ffn, S);
            before = &W.st_ffn;
        }
        CERA_TRY(layered_alloc(m, static_cast<uint64_t>(W.attn.kv_heads) * g.cap * W.attn.row * g.esz, &W.kv, true));
        proj = std::max<uint64_t>(proj, dense_pad(W.in.rows));
        att = std::max<uint64_t>(att, W.o.kp);
        q = std::max<uint64_t>(q, static_cast<uint64_t>(a.heads) * W.attn.kp);
        ff = std::max<uint64_t>(ff, W.down.kp);
        if (W.latent) lat = std::max<uint64_t>(lat, static_cast<uint64_t>(a.heads) * W.attn.vp);
        widest = std::max({widest, att, ff});
    }
    std::fill(before->next, before->next + S, 1.0f);   // the sum of the streams leaves the last layer
    CERA_TRY(layered_alloc_t(m, S * ld, &g.x));
    CERA_TRY(layered_alloc_t(m, ld, &g.u));
    CERA_TRY(layered_alloc_t(m, proj, &g.qkvg));
    if (first) CERA_TRY(layered_alloc_t(m, first, &g.v_first));
    CERA_TRY(layered_alloc(m, q * g.esz, &g.q, true));
    CERA_TRY(layered_alloc(m, att * g.esz, &g.cat, true));
    if (ff) CERA_TRY(layered_alloc(m, ff * g.esz, &g.act, true));
    if (lat) CERA_TRY(layered_alloc(m, lat * g.esz, &g.lat, true));
    m->hidden = g.u;
    g.step_fits = cera_dense_gemv_fits(widest, g.f32);
    return CERA_HIP_OK;
}
