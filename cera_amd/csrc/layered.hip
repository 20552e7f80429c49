// The layered float model family (cera_hip_layered_create), parallel blocks: weights in HBM, the per-layer state (KV
// cache and convolution ring of every pass over a layer), the decode step and the batched pass; and what parallel
// and sequential blocks share.
//
// Decode, per layer, three launches: [norm, both input convolutions, Q|K|V|gate and gate|up
// with SwiGLU] - [rotation, append, attention, head gates; the convolutions' history for the next
// token beside it] - [O and down as one product over the two inputs side by side, added to the
// residual; it also adds up attention's partial results over key ranges].  A very long key range adds
// a launch for that sum.
#include <algorithm>
#include <cmath>
#include <cstring>
#include <new>

#include "layered.h"

namespace {

constexpr uint32_t RING_DEPTH = 64;   // rows a convolution ring keeps: how far a sequence can be cut back

}  // namespace

cera_hip_status layered_alloc(cera_hip_model* m, uint64_t bytes, void** out, bool zero) {
    *out = nullptr;
    HIP_TRY(m->ctx, hipMalloc(out, bytes ? bytes : 256));
    m->owned.push_back(*out);
    m->bytes += bytes;
    if (zero) HIP_TRY(m->ctx, hipMemsetAsync(*out, 0, bytes, m->ctx->stream));
    return CERA_HIP_OK;
}
cera_hip_status layered_put_vec(cera_hip_model* m, const float* src, uint64_t n, uint64_t ld, float** out) {
    std::vector<float> v(ld, 0.0f);
    std::copy(src, src + n, v.begin());
    CERA_TRY(layered_alloc_t(m, ld, out, false));
    return cera_hip_upload(m->ctx, *out, v.data(), ld * 4);
}
void Packer::row(uint64_t dst, uint64_t col, const cera_hip_tensor& t, uint64_t src, uint64_t c0, uint64_t n) {
    std::memcpy(host.data() + dst * kp + col, static_cast<const uint16_t*>(t.data) + src * t.k + c0, (n ? n : t.k) * 2);
}
void Packer::rows(uint64_t dst, uint64_t col, const cera_hip_tensor& t) {
    for (uint64_t r = 0; r < t.m; ++r) row(dst + r, col, t, r);
}
cera_hip_status Packer::put(cera_hip_model* m, DenseMat* out) {
    out->kp = static_cast<uint32_t>(kp);
    out->rows = static_cast<uint32_t>(host.size() / kp);
    CERA_TRY(layered_alloc(m, host.size() * 2, &out->w, false));
    return cera_hip_upload(m->ctx, out->w, host.data(), host.size() * 2);
}
float layered_get(const CeraLayered& g, const void* rows, uint64_t i) {
    if (g.f32) return static_cast<const float*>(rows)[i];
    const uint32_t b = static_cast<uint32_t>(static_cast<const uint16_t*>(rows)[i]) << 16;
    float f;
    std::memcpy(&f, &b, 4);
    return f;
}
void layered_set(const CeraLayered& g, void* rows, uint64_t i, float f) {
    if (g.f32) { static_cast<float*>(rows)[i] = f; return; }
    uint32_t b;
    std::memcpy(&b, &f, 4);
    static_cast<uint16_t*>(rows)[i] = static_cast<uint16_t>((b + 0x7FFFu + ((b >> 16) & 1)) >> 16);   // nearest even
}
void layered_batch_free(cera_hip_model* m) {
    CeraLayered& g = *m->layered;
    for (void* p : g.b_owned) (void)hipFree(p);
    g.b_owned.clear();
    m->bytes -= std::min(m->bytes, g.b_bytes);
    g.b_bytes = 0;
    g.cap_n = g.logits_cap = 0;
    g.blogits = nullptr;
}
cera_hip_status layered_batch_alloc(cera_hip_model* m, uint64_t bytes, void** out) {
    CeraLayered& g = *m->layered;
    *out = nullptr;
    HIP_TRY(m->ctx, hipMalloc(out, bytes));
    g.b_owned.push_back(*out);
    g.b_bytes += bytes;
    m->bytes += bytes;
    // pad columns are read by the products, against zero weights: they have to be finite
    HIP_TRY(m->ctx, hipMemsetAsync(*out, 0, bytes, m->ctx->stream));
    return CERA_HIP_OK;
}
cera_hip_status layered_batch_logits(cera_hip_model* m, uint32_t n) {
    CeraLayered& g = *m->layered;
    if (g.logits_cap >= n) return CERA_HIP_OK;   // grows with the pass buffers only: an older, smaller one is freed with them
    CERA_TRY(layered_batch_alloc(m, static_cast<uint64_t>(g.cap_n) * g.cfg.vocab * 4, reinterpret_cast<void**>(&g.blogits)));
    g.logits_cap = g.cap_n;
    return CERA_HIP_OK;
}
cera_hip_status layered_portions(cera_hip_model* m, LayeredPass pass, const uint32_t* tokens, uint32_t n, uint32_t start, float* last_logits, float* all) {
    if (n == 1) {
        CERA_TRY(m->ops->decode(m, tokens[0], start, true));
        m->seq_len = start + 1;
        return cera_hip_download(m->ctx, all ? all : last_logits, m->logits, static_cast<uint64_t>(m->cfg.vocab) * 4);
    }
    for (uint32_t off = 0; off < n; off += CERA_PREFILL_CHUNK) {
        const uint32_t len = std::min(CERA_PREFILL_CHUNK, n - off);
        CERA_TRY(pass(m, tokens + off, len, start + off, !all && off + len == n, all ? all + static_cast<uint64_t>(off) * m->cfg.vocab : nullptr));
        m->seq_len = start + off + len;
    }
    return all ? CERA_HIP_OK : cera_hip_download(m->ctx, last_logits, m->logits, static_cast<uint64_t>(m->cfg.vocab) * 4);
}

namespace {

using L = CeraLayered;

// Per-pair (cos, sin) of every position.  Frequencies base^(-2 i / dims); with yarn the low ones are
// divided by the factor, the high ones kept, blended linearly between the dimensions that turn `fast`
// and `slow` times over the original length, and both values scaled by 0.1 ln(factor) + 1.
std::vector<float> rotation_table(const cera_hip_attn_spec& s, uint32_t positions) {
    const uint32_t half = s.rot_dims / 2;
    std::vector<double> f(half);
    double mag = 1.0;
    for (uint32_t i = 0; i < half; ++i) f[i] = std::pow(s.rot_base, -2.0 * i / s.rot_dims);
    if (s.yarn) {
        const double pi = 3.14159265358979323846;
        auto dim_of = [&](double turns) { return s.rot_dims * std::log(s.yarn_original / (2 * pi * turns)) / (2 * std::log(s.rot_base)); };
        const double lo = std::max(std::floor(dim_of(s.yarn_fast)), 0.0);
        const double hi = std::min(std::ceil(dim_of(s.yarn_slow)), static_cast<double>(s.rot_dims) - 1.0);
        for (uint32_t i = 0; i < half; ++i) {
            const double ramp = std::min(std::max((i - lo) / std::max(hi - lo, 0.001), 0.0), 1.0);
            f[i] = f[i] / s.yarn_factor * ramp + f[i] * (1.0 - ramp);
        }
        mag = 0.1 * std::log(s.yarn_factor) + 1.0;
    }
    std::vector<float> t(static_cast<uint64_t>(positions) * s.rot_dims);
    for (uint32_t p = 0; p < positions; ++p)
        for (uint32_t i = 0; i < half; ++i) {
            t[static_cast<uint64_t>(p) * s.rot_dims + 2 * i] = static_cast<float>(std::cos(p * f[i]) * mag);
            t[static_cast<uint64_t>(p) * s.rot_dims + 2 * i + 1] = static_cast<float>(std::sin(p * f[i]) * mag);
        }
    return t;
}

}  // namespace

cera_hip_status layered_rotation(cera_hip_model* m, const cera_hip_attn_spec& s, RotationTables* tables, const float** out) {
    if (!s.rot_dims) return CERA_HIP_OK;
    float*& t = (*tables)[std::make_tuple(s.rot_dims, s.rot_base, s.yarn, s.yarn_factor, s.yarn_original, s.yarn_fast, s.yarn_slow)];
    if (!t) {
        const std::vector<float> host = rotation_table(s, m->layered->cap);
        CERA_TRY(layered_put_vec(m, host.data(), host.size(), host.size(), &t));
    }
    *out = t;
    return CERA_HIP_OK;
}

namespace {

// ---- the decode step ------------------------------------------------------------------------------
cera_hip_status batch_pass(cera_hip_model* m, const uint32_t* tokens, uint32_t n, uint32_t start, bool last, float* all);

void advance_ring(L& g, uint32_t start, uint32_t end) {
    if (start == 0) g.ring_lo = 0;
    g.ring_lo = std::max(g.ring_lo, end > RING_DEPTH ? end - RING_DEPTH : 0u);
}
float* ring_row(const ConvRing& r, uint32_t pos) { return r.rows + static_cast<uint64_t>(pos & (r.depth - 1)) * r.ld; }

SAttnPass step_pass(const L& g, const LayerW& W, const Run& R, uint32_t pos) {
    SAttnPass p;
    p.qkvg = g.qkvg; p.ld = dense_pad(W.qkvg.rows); p.n = 1; p.start = pos;
    p.kc = R.kc; p.vc = R.vc; p.cap = g.cap; p.q = g.q; p.out = g.cat; p.out_ld = W.down.kp;
    return p;
}

cera_hip_status decode(cera_hip_model* m, uint32_t token, uint32_t pos, bool want_logits) {
    L& g = *m->layered;
    cera_hip_ctx* ctx = m->ctx;
    if (!g.step_fits) return batch_pass(m, &token, 1, pos, want_logits, nullptr);
    const uint32_t width = g.cfg.width;
    auto gemv = [&](const DenseIn& in, const DenseMat& wa, const DenseOut& oa, const DenseMat* wb = nullptr, const DenseOut* ob = nullptr) {
        bool ok = false;
        cera_hip_status st = cera_launch_dense_gemv(ctx, in, wa, oa, wb, ob, g.f32, &ok);
        if (st == CERA_HIP_OK && !ok) st = cera_fail(ctx, CERA_HIP_ERR_SHAPE, "decode: a product's input does not fit the GEMV");
        return st;
    };
    CERA_TRY(cera_launch_embed_pos(ctx, g.embed, g.pos, nullptr, token, 1, pos, width, g.ld, g.x, g.x0));
    for (Run& R : g.runs) {
        const LayerW& W = g.layers[R.layer];
        if (R.step >= 0) {
            DenseIn in;
            in.kind = DenseIn::CONCAT; in.x = g.x; in.x2 = g.x0;
            DenseOut out;
            out.out = g.xb; out.bias = g.loop_step + R.step * g.ld; out.rows = width;
            CERA_TRY(gemv(in, g.loop_in, out));
            std::swap(g.x, g.xb);
        }
        if (R.ring.rows && g.hist_pos != pos) CERA_TRY(cera_launch_conv_hist(ctx, R.ring, R.hist, pos));
        DenseIn in;
        in.kind = DenseIn::NORM; in.x = g.x; in.n_mean = width; in.eps = g.cfg.eps;
        in.scale_a = W.scale_a; in.scale_b = W.scale_b;
        if (R.ring.rows) {
            in.add_a = R.hist.a; in.add_b = R.hist.b;
            in.plain = W.norm; in.h_out = ring_row(R.ring, pos);
        }
        DenseOut oq, of;
        oq.out = g.qkvg; oq.rows = W.qkvg.rows;
        of.epi = DENSE_SWIGLU; of.rows = W.ff;
        of.out = static_cast<char*>(g.cat) + W.att_p * g.esz;
        CERA_TRY(gemv(in, W.qkvg, oq, W.ff ? &W.gate_up : nullptr, &of));
        DenseIn raw;
        raw.x = g.cat;
        CERA_TRY(cera_launch_sattn_step(ctx, W.shape, step_pass(g, W, R, pos), R.ring, R.hist, &raw.merge, g.f32));
        if (raw.merge.part) raw.kind = DenseIn::MERGE;
        DenseOut add;
        add.epi = DENSE_ADD; add.out = g.x; add.mult = g.cfg.residual_mult; add.rows = width;
        CERA_TRY(gemv(raw, W.down, add));
    }
    g.hist_pos = pos + 1;
    advance_ring(g, pos, pos + 1);
    m->hidden = g.x;
    if (want_logits) {
        DenseIn in;
        in.kind = DenseIn::NORM; in.x = g.x; in.n_mean = width; in.eps = g.cfg.eps; in.scale_a = g.final_norm;
        DenseOut out;
        out.out = m->logits; out.rows = g.cfg.vocab;
        CERA_TRY(gemv(in, g.head, out));
    }
    return CERA_HIP_OK;
}

// ---- the batched pass -----------------------------------------------------------------------------
cera_hip_status ensure_batch(cera_hip_model* m, uint32_t n, bool logits) {
    L& g = *m->layered;
    const uint32_t limit = std::min<uint32_t>(CERA_PREFILL_CHUNK, g.cfg.max_seq_len);
    if (g.cap_n < n) {
        HIP_TRY(m->ctx, hipStreamSynchronize(m->ctx->stream));
        layered_batch_free(m);
        const uint64_t N = std::min<uint64_t>(limit, (n + 255) / 256 * 256);
        uint64_t qkvg = 0, cat = 0, q = 0;
        for (const LayerW& W : g.layers) {
            qkvg = std::max<uint64_t>(qkvg, dense_pad(W.qkvg.rows));
            cat = std::max<uint64_t>(cat, W.down.kp);
            q = std::max<uint64_t>(q, static_cast<uint64_t>(W.shape.heads) * sattn_pad32(W.shape.dim));
        }
        auto all = [&]() -> cera_hip_status {
            auto fl = [&](uint64_t n_el, float** p) { return layered_batch_alloc(m, n_el * 4, reinterpret_cast<void**>(p)); };
            CERA_TRY(fl(N * g.ld, &g.bx));
            CERA_TRY(fl(N * g.ld, &g.bx0));
            CERA_TRY(fl(N * qkvg, &g.bqkvg));
            CERA_TRY(fl(N, &g.binv));
            CERA_TRY(layered_batch_alloc(m, N * g.ld * g.esz, &g.ba));
            CERA_TRY(layered_batch_alloc(m, N * g.ld * g.esz, &g.bb));
            CERA_TRY(layered_batch_alloc(m, N * q * g.esz, &g.bq));
            CERA_TRY(layered_batch_alloc(m, N * cat * g.esz, &g.bcat));
            if (g.loop_in.w) CERA_TRY(layered_batch_alloc(m, N * 2 * g.ld * g.esz, &g.bcat2));
            return layered_batch_alloc(m, N * 4, reinterpret_cast<void**>(&g.btok));
        };
        const cera_hip_status st = all();
        if (st != CERA_HIP_OK) { layered_batch_free(m); return st; }
        g.cap_n = static_cast<uint32_t>(N);
    }
    if (logits) CERA_TRY(layered_batch_logits(m, n));
    return CERA_HIP_OK;
}

// n tokens (at most CERA_PREFILL_CHUNK) from `start`; `last`: the last position's logits into m->logits;
// all (nullable): every position's logits, host
cera_hip_status batch_pass(cera_hip_model* m, const uint32_t* tokens, uint32_t n, uint32_t start, bool last, float* all) {
    L& g = *m->layered;
    cera_hip_ctx* ctx = m->ctx;
    const uint32_t width = g.cfg.width;
    CERA_TRY(ensure_batch(m, n, all != nullptr));
    CERA_TRY(cera_hip_upload(ctx, g.btok, tokens, n * 4ull));
    CERA_TRY(cera_launch_embed_pos(ctx, g.embed, g.pos, g.btok, 0, n, start, width, g.ld, g.bx, g.bx0));
    for (const Run& R : g.runs) {
        const LayerW& W = g.layers[R.layer];
        if (R.step >= 0) {
            CERA_TRY(cera_launch_concat2(ctx, g.bx, g.bx0, n, g.ld, g.bcat2, g.f32));
            DenseOut out;
            out.out = g.bx; out.ld = g.ld; out.bias = g.loop_step + R.step * g.ld; out.rows = width;
            CERA_TRY(cera_launch_dense_gemm(ctx, g.loop_in, g.bcat2, 2 * g.ld, n, out, g.f32));
        }
        NormConv nc;
        nc.x = g.bx; nc.ld = g.ld; nc.n = n; nc.start = start; nc.width = width; nc.taps = g.cfg.conv_taps; nc.eps = g.cfg.eps;
        nc.w = W.norm; nc.wa = W.conv_a; nc.wb = W.conv_b; nc.ring = R.ring;
        nc.out_a = g.ba; nc.out_b = W.ff ? g.bb : nullptr; nc.inv = g.binv;
        CERA_TRY(cera_launch_norm_conv(ctx, nc, g.f32));
        DenseOut oq;
        oq.out = g.bqkvg; oq.ld = dense_pad(W.qkvg.rows); oq.rows = W.qkvg.rows;
        CERA_TRY(cera_launch_dense_gemm(ctx, W.qkvg, g.ba, g.ld, n, oq, g.f32));
        if (W.ff) {
            DenseOut of;
            of.epi = DENSE_SWIGLU; of.rows = W.ff; of.ld = W.down.kp;
            of.out = static_cast<char*>(g.bcat) + W.att_p * g.esz;
            CERA_TRY(cera_launch_dense_gemm(ctx, W.gate_up, g.bb, g.ld, n, of, g.f32));
        }
        SAttnPass p;
        p.qkvg = g.bqkvg; p.ld = oq.ld; p.n = n; p.start = start;
        p.kc = R.kc; p.vc = R.vc; p.cap = g.cap; p.q = g.bq; p.out = g.bcat; p.out_ld = W.down.kp;
        CERA_TRY(cera_launch_sattn_append(ctx, W.shape, p, R.ring, g.bx, g.ld, g.binv, W.norm, g.f32));
        CERA_TRY(cera_launch_sattn(ctx, W.shape, p, g.f32));
        DenseOut add;
        add.epi = DENSE_ADD; add.out = g.bx; add.ld = g.ld; add.mult = g.cfg.residual_mult; add.rows = width;
        CERA_TRY(cera_launch_dense_gemm(ctx, W.down, g.bcat, W.down.kp, n, add, g.f32));
    }
    g.hist_pos = UINT32_MAX;
    advance_ring(g, start, start + n);
    m->hidden = g.bx + static_cast<uint64_t>(n - 1) * g.ld;
    if (!last && !all) return CERA_HIP_OK;
    NormConv nc;
    nc.x = all ? g.bx : m->hidden; nc.ld = g.ld; nc.n = all ? n : 1; nc.width = width; nc.eps = g.cfg.eps; nc.w = g.final_norm; nc.out_a = g.ba;
    CERA_TRY(cera_launch_norm_conv(ctx, nc, g.f32));
    DenseOut out;
    out.out = all ? g.blogits : m->logits; out.ld = g.cfg.vocab; out.rows = g.cfg.vocab;
    CERA_TRY(cera_launch_dense_gemm(ctx, g.head, g.ba, g.ld, nc.n, out, g.f32));
    return all ? cera_hip_download(ctx, all, g.blogits, static_cast<uint64_t>(n) * g.cfg.vocab * 4) : CERA_HIP_OK;
}

cera_hip_status prefill(cera_hip_model* m, const uint32_t* tokens, uint32_t n, uint32_t start, float* last_logits) {
    return layered_portions(m, batch_pass, tokens, n, start, last_logits, nullptr);
}
cera_hip_status prefill_all(cera_hip_model* m, const uint32_t* tokens, uint32_t n, uint32_t start, float* logits) {
    return layered_portions(m, batch_pass, tokens, n, start, nullptr, logits);
}

// ---- state ----------------------------------------------------------------------------------------
uint32_t conv_first(const L& g, uint32_t len) {   // oldest position the token at `len` reads through a convolution
    const uint32_t back = g.cfg.conv_taps - 1;
    return len > back ? len - back : 0;
}
cera_hip_status truncate(cera_hip_model* m, uint32_t len) {
    L& g = *m->layered;
    if (len && g.cfg.conv_taps > 1 && conv_first(g, len) < g.ring_lo)
        return cera_fail(m->ctx, CERA_HIP_ERR_POSITION, "truncate: the convolution state reaches back to position " + std::to_string(g.ring_lo) +
                                                            " only; cannot continue from " + std::to_string(len));
    return CERA_HIP_OK;
}

// cache rows <-> time-major f32 [n][kv_heads * dim] / [n][kv_heads * vdim]
cera_hip_status move_kv(cera_hip_model* m, uint32_t run, float* k, float* v, uint32_t n, bool read) {
    L& g = *m->layered;
    const Run& R = g.runs[run];
    const SAttnShape& s = g.layers[R.layer].shape;
    const uint64_t dp = sattn_pad32(s.dim), vp = sattn_pad32(s.vdim);
    std::vector<char> rows;
    auto get = [&](uint64_t i) { return layered_get(g, rows.data(), i); };
    auto set = [&](uint64_t i, float f) { layered_set(g, rows.data(), i, f); };
    for (uint32_t h = 0; h < s.kv_heads && n; ++h) {
        char* const kd = static_cast<char*>(R.kc) + static_cast<uint64_t>(h) * g.cap * dp * g.esz;
        rows.assign(static_cast<uint64_t>(n) * dp * g.esz, 0);
        if (read) CERA_TRY(cera_hip_download(m->ctx, rows.data(), kd, rows.size()));
        for (uint32_t t = 0; t < n; ++t)
            for (uint32_t c = 0; c < s.dim; ++c) {
                float& f = k[(static_cast<uint64_t>(t) * s.kv_heads + h) * s.dim + c];
                if (read) f = get(t * dp + c); else set(t * dp + c, f);
            }
        if (!read) CERA_TRY(cera_hip_upload(m->ctx, kd, rows.data(), rows.size()));
        char* const vd = static_cast<char*>(R.vc) + static_cast<uint64_t>(h) * vp * g.cap * g.esz;
        rows.assign(static_cast<uint64_t>(s.vdim) * g.cap * g.esz, 0);
        if (read) CERA_TRY(cera_hip_download(m->ctx, rows.data(), vd, rows.size()));
        for (uint32_t c = 0; c < s.vdim; ++c)
            for (uint32_t t = 0; t < n; ++t) {
                float& f = v[(static_cast<uint64_t>(t) * s.kv_heads + h) * s.vdim + c];
                if (read) f = get(static_cast<uint64_t>(c) * g.cap + t); else set(static_cast<uint64_t>(c) * g.cap + t, f);
            }
        if (!read) CERA_TRY(cera_hip_upload(m->ctx, vd, rows.data(), rows.size()));
    }
    return CERA_HIP_OK;
}
cera_hip_status read_kv(cera_hip_model* m, uint32_t run, float* k, float* v) { return move_kv(m, run, k, v, m->seq_len, true); }
cera_hip_status write_kv(cera_hip_model* m, uint32_t run, const float* k, const float* v, uint32_t n) {
    return move_kv(m, run, const_cast<float*>(k), const_cast<float*>(v), n, false);
}

cera_hip_status read_conv(cera_hip_model* m, uint32_t run, float* rows) {
    L& g = *m->layered;
    const Run& R = g.runs[run];
    const uint32_t back = g.cfg.conv_taps - 1, width = g.cfg.width;
    for (uint32_t j = 0; j < back; ++j) {
        float* dst = rows + static_cast<uint64_t>(j) * width;
        if (m->seq_len + j < back) std::fill(dst, dst + width, 0.0f);
        else CERA_TRY(cera_hip_download(m->ctx, dst, ring_row(R.ring, m->seq_len + j - back), width * 4ull));
    }
    return CERA_HIP_OK;
}
cera_hip_status write_conv(cera_hip_model* m, uint32_t run, const float* rows, uint32_t n) {
    L& g = *m->layered;
    const Run& R = g.runs[run];
    const uint32_t back = g.cfg.conv_taps - 1, width = g.cfg.width;
    for (uint32_t j = 0; j < back; ++j)
        if (n + j >= back) CERA_TRY(cera_hip_upload(m->ctx, ring_row(R.ring, n + j - back), rows + static_cast<uint64_t>(j) * width, width * 4ull));
    g.ring_lo = conv_first(g, n);
    g.hist_pos = UINT32_MAX;
    return CERA_HIP_OK;
}

const CeraModelOps OPS = {decode, prefill, prefill_all, truncate, read_kv, write_kv, read_conv, write_conv, layered_destroy};

}  // namespace

void layered_destroy(cera_hip_model* m) {
    cera_hip_ctx* ctx = m->ctx;
    std::lock_guard<std::recursive_mutex> lk(ctx->op_mu);
    (void)hipStreamSynchronize(ctx->stream);
    if (m->layered) {
        for (void* p : m->layered->b_owned) (void)hipFree(p);
        delete m->layered;
    }
    for (void* p : m->owned)
        if (p) (void)hipFree(p);
    delete m;
}
cera_hip_status layered_bad(cera_hip_ctx* ctx, const std::string& what) { return cera_fail(ctx, CERA_HIP_ERR_SHAPE, "layered_create: " + what); }
cera_hip_status layered_mat(cera_hip_ctx* ctx, const cera_hip_tensor& t, uint64_t m, uint64_t k, const char* name) {
    if (t.ggml_type != CERA_HIP_BF16)
        return cera_fail(ctx, CERA_HIP_ERR_UNSUPPORTED_DTYPE, std::string(name) + ": the layered family takes bf16 matrices");
    if (!t.data || t.m != m || t.k != k || t.nbytes != m * k * 2)
        return layered_bad(ctx, std::string(name) + ": expected [" + std::to_string(m) + " x " + std::to_string(k) + "], got [" + std::to_string(t.m) +
                                    " x " + std::to_string(t.k) + "]");
    return CERA_HIP_OK;
}

namespace {

cera_hip_status check(cera_hip_ctx* ctx, const cera_hip_layered_config& c, const cera_hip_layered_layer* layers) {
    auto bad = [&](const std::string& what) { return layered_bad(ctx, what); };
    if (c.block == CERA_HIP_BLOCK_SEQUENTIAL) return layered_seq_check(ctx, c, layers);
    if (c.block != CERA_HIP_BLOCK_PARALLEL) return bad("unknown block form");
    if (!c.n_layers || !c.width || !c.vocab || !c.max_seq_len || !c.conv_taps) return bad("zero dimension in config");
    if (c.conv_taps > CONV_MAX_TAPS) return bad("conv_taps above " + std::to_string(CONV_MAX_TAPS));
    if (!c.final_norm) return cera_fail(ctx, CERA_HIP_ERR_ARGUMENT, "layered_create: final_norm missing");
    auto mat = [&](const cera_hip_tensor& t, uint64_t rows, uint64_t k, const char* name) { return layered_mat(ctx, t, rows, k, name); };
    CERA_TRY(mat(c.embed, c.vocab, c.width, "embed"));
    CERA_TRY(mat(c.head, c.vocab, c.width, "head"));
    if (c.pos.m < c.max_seq_len) return bad("pos has fewer rows than max_seq_len");
    CERA_TRY(mat(c.pos, c.pos.m, c.width, "pos"));
    if (c.loop_times) {
        if (c.loop_start >= c.loop_stop || c.loop_stop > c.n_layers) return bad("loop range");
        if (!c.loop_step) return cera_fail(ctx, CERA_HIP_ERR_ARGUMENT, "layered_create: loop_step missing");
        CERA_TRY(mat(c.loop_in, c.width, 2ull * c.width, "loop_in"));
    }
    for (uint32_t i = 0; i < c.n_layers; ++i) {
        const cera_hip_layered_layer& Y = layers[i];
        const cera_hip_attn_spec& a = Y.attn;
        if (a.kind != CERA_HIP_MIXER_SIGMOID) return bad("layer " + std::to_string(i) + ": parallel blocks take the sigmoid mixer");
        if (!a.heads || !a.kv_heads || a.heads % a.kv_heads || !a.dim || !a.vdim || a.dim > 256 || a.vdim > 256)
            return bad("layer " + std::to_string(i) + ": heads must be a multiple of kv_heads, head sizes at most 256");
        if (a.rot_dims % 2 || a.rot_dims > a.dim) return bad("layer " + std::to_string(i) + ": rot_dims must be even and at most dim");
        if (!Y.norm || !Y.conv_attn || !Y.score_bias || (Y.ff && !Y.conv_ffn))
            return cera_fail(ctx, CERA_HIP_ERR_ARGUMENT, "layered_create: layer vectors missing");
        CERA_TRY(mat(Y.q, static_cast<uint64_t>(a.heads) * a.dim, c.width, "q"));
        CERA_TRY(mat(Y.k, static_cast<uint64_t>(a.kv_heads) * a.dim, c.width, "k"));
        CERA_TRY(mat(Y.v, static_cast<uint64_t>(a.kv_heads) * a.vdim, c.width, "v"));
        CERA_TRY(mat(Y.head_gate, a.heads, c.width, "head_gate"));
        CERA_TRY(mat(Y.o, c.width, static_cast<uint64_t>(a.heads) * a.vdim, "o"));
        if (Y.ff) {
            CERA_TRY(mat(Y.ffn_gate, Y.ff, c.width, "ffn_gate"));
            CERA_TRY(mat(Y.ffn_up, Y.ff, c.width, "ffn_up"));
            CERA_TRY(mat(Y.ffn_down, c.width, Y.ff, "ffn_down"));
        }
    }
    return CERA_HIP_OK;
}

cera_hip_status build(cera_hip_model* m, const cera_hip_layered_config& c, const cera_hip_layered_layer* layers) {
    L& g = *m->layered;
    cera_hip_ctx* ctx = m->ctx;
    g.ld = dense_pad(c.width);
    g.cap = (c.max_seq_len + SATTN_CAP_STEP - 1) / SATTN_CAP_STEP * SATTN_CAP_STEP;
    g.f32 = c.f32 != 0;
    g.esz = g.f32 ? 4 : 2;
    const uint64_t ld = g.ld;
    // tables of bf16 rows, as they are
    auto table = [&](const cera_hip_tensor& t, void** out) -> cera_hip_status {
        CERA_TRY(layered_alloc(m, t.nbytes, out, false));
        return cera_hip_upload(ctx, *out, t.data, t.nbytes);
    };
    CERA_TRY(table(c.embed, &g.embed));
    {
        Packer p(c.vocab, ld);
        p.rows(0, 0, c.head);
        CERA_TRY(p.put(m, &g.head));
    }
    CERA_TRY(layered_put_vec(m, c.final_norm, c.width, ld, &g.final_norm));
    CERA_TRY(layered_alloc_t(m, dense_pad(c.vocab), &m->logits));
    CERA_TRY(layered_alloc_t(m, 4, &m->scalars));
    if (c.block == CERA_HIP_BLOCK_SEQUENTIAL) return layered_seq_build(m, c, layers);
    CERA_TRY(table(c.pos, &g.pos));
    if (c.loop_times) {
        Packer p(c.width, 2 * ld);
        for (uint32_t r = 0; r < c.width; ++r) {
            p.row(r, 0, c.loop_in, r, 0, c.width);
            p.row(r, ld, c.loop_in, r, c.width, c.width);
        }
        CERA_TRY(p.put(m, &g.loop_in));
        std::vector<float> st(c.loop_times * ld, 0.0f);
        for (uint32_t t = 0; t < c.loop_times; ++t) std::copy(c.loop_step + static_cast<uint64_t>(t) * c.width, c.loop_step + static_cast<uint64_t>(t + 1) * c.width, st.begin() + t * ld);
        CERA_TRY(layered_put_vec(m, st.data(), st.size(), st.size(), &g.loop_step));
    }
    RotationTables tables;   // shared between layers
    uint64_t max_qkvg = 0, max_cat = 0, max_q = 0;
    g.layers.resize(c.n_layers);
    for (uint32_t i = 0; i < c.n_layers; ++i) {
        const cera_hip_layered_layer& Y = layers[i];
        const cera_hip_attn_spec& a = Y.attn;
        LayerW& W = g.layers[i];
        SAttnShape& s = W.shape;
        s.heads = a.heads; s.kv_heads = a.kv_heads; s.dim = a.dim; s.vdim = a.vdim; s.chunk = a.chunk; s.scale = a.scale; s.rot_dims = a.rot_dims;
        CERA_TRY(layered_rotation(m, a, &tables, &s.rot_table));
        float* bias;
        CERA_TRY(layered_put_vec(m, Y.score_bias, a.heads, a.heads, &bias));
        s.bias = bias;
        {
            Packer p(Y.q.m + Y.k.m + Y.v.m + Y.head_gate.m, ld);
            p.rows(0, 0, Y.q);
            p.rows(Y.q.m, 0, Y.k);
            p.rows(Y.q.m + Y.k.m, 0, Y.v);
            p.rows(Y.q.m + Y.k.m + Y.v.m, 0, Y.head_gate);
            CERA_TRY(p.put(m, &W.qkvg));
        }
        W.ff = Y.ff;
        W.att_p = dense_pad(Y.o.k);
        Packer pd(c.width, W.att_p + (Y.ff ? dense_pad(Y.ff) : 0));
        pd.rows(0, 0, Y.o);
        if (Y.ff) {
            const uint64_t groups = (Y.ff + 15) / 16;
            Packer p(groups * 32, ld);   // 16 gate rows, their 16 up rows, ...
            for (uint32_t r = 0; r < Y.ff; ++r) {
                p.row((r >> 4) * 32 + (r & 15), 0, Y.ffn_gate, r);
                p.row((r >> 4) * 32 + 16 + (r & 15), 0, Y.ffn_up, r);
            }
            CERA_TRY(p.put(m, &W.gate_up));
            pd.rows(0, W.att_p, Y.ffn_down);
        }
        CERA_TRY(pd.put(m, &W.down));
        CERA_TRY(layered_put_vec(m, Y.norm, c.width, ld, &W.norm));
        auto conv = [&](const float* src, float** taps_out, float** scale_out) -> cera_hip_status {
            std::vector<float> t(c.conv_taps * ld, 0.0f), sc(ld, 0.0f);
            for (uint32_t ch = 0; ch < c.width; ++ch) {
                for (uint32_t j = 0; j < c.conv_taps; ++j) t[j * ld + ch] = src[static_cast<uint64_t>(ch) * c.conv_taps + j];
                sc[ch] = Y.norm[ch] * (1.0f + src[static_cast<uint64_t>(ch) * c.conv_taps + c.conv_taps - 1]);
            }
            CERA_TRY(layered_put_vec(m, t.data(), t.size(), t.size(), taps_out));
            return layered_put_vec(m, sc.data(), ld, ld, scale_out);
        };
        CERA_TRY(conv(Y.conv_attn, &W.conv_a, &W.scale_a));
        if (Y.ff) CERA_TRY(conv(Y.conv_ffn, &W.conv_b, &W.scale_b));
        max_qkvg = std::max<uint64_t>(max_qkvg, dense_pad(W.qkvg.rows));
        max_cat = std::max<uint64_t>(max_cat, W.down.kp);
        max_q = std::max<uint64_t>(max_q, static_cast<uint64_t>(a.heads) * sattn_pad32(a.dim));
    }
    // execution order
    auto add_run = [&](uint32_t layer, int step) { Run r; r.layer = layer; r.step = step; g.runs.push_back(r); };
    for (uint32_t i = 0; i < c.n_layers;) {
        if (c.loop_times && i == c.loop_start) {
            for (uint32_t t = 0; t < c.loop_times; ++t)
                for (uint32_t j = c.loop_start; j < c.loop_stop; ++j) add_run(j, j == c.loop_start ? static_cast<int>(t) : -1);
            i = c.loop_stop;
        } else {
            add_run(i++, -1);
        }
    }
    for (Run& R : g.runs) {
        const LayerW& W = g.layers[R.layer];
        const SAttnShape& s = W.shape;
        CERA_TRY(layered_alloc(m, static_cast<uint64_t>(s.kv_heads) * g.cap * sattn_pad32(s.dim) * g.esz, &R.kc, true));
        CERA_TRY(layered_alloc(m, static_cast<uint64_t>(s.kv_heads) * g.cap * sattn_pad32(s.vdim) * g.esz, &R.vc, true));
        if (c.conv_taps > 1) {
            R.ring.depth = RING_DEPTH; R.ring.ld = ld; R.ring.width = static_cast<uint32_t>(ld);
            CERA_TRY(layered_alloc_t(m, RING_DEPTH * ld, &R.ring.rows));
            R.hist.wa = W.conv_a; R.hist.wb = W.conv_b; R.hist.taps = c.conv_taps;
            CERA_TRY(layered_alloc_t(m, ld, &R.hist.a));
            CERA_TRY(layered_alloc_t(m, ld, &R.hist.b));
        }
    }
    CERA_TRY(layered_alloc_t(m, ld, &g.x));
    CERA_TRY(layered_alloc_t(m, ld, &g.xb));
    CERA_TRY(layered_alloc_t(m, ld, &g.x0));
    CERA_TRY(layered_alloc_t(m, max_qkvg, &g.qkvg));
    CERA_TRY(layered_alloc(m, max_q * g.esz, &g.q, true));
    CERA_TRY(layered_alloc(m, max_cat * g.esz, &g.cat, true));
    m->hidden = g.x;
    const uint64_t widest = std::max<uint64_t>(max_cat, (c.loop_times ? 2 : 1) * ld);
    g.step_fits = cera_dense_gemv_fits(widest, g.f32);
    return CERA_HIP_OK;
}

}  // namespace

extern "C" cera_hip_status cera_hip_layered_create(cera_hip_ctx* ctx, const cera_hip_layered_config* cfg,
                                                   const cera_hip_layered_layer* layers, cera_hip_model** out) {
    if (!ctx || !cfg || !layers || !out) return CERA_HIP_ERR_ARGUMENT;
    std::lock_guard<std::recursive_mutex> lk(ctx->op_mu);
    *out = nullptr;
    CERA_TRY(check(ctx, *cfg, layers));
    cera_hip_model* m = new (std::nothrow) cera_hip_model();
    if (!m) return cera_fail(ctx, CERA_HIP_ERR_OOM, "host allocation failed");
    m->ctx = ctx;
    m->ops = cfg->block == CERA_HIP_BLOCK_SEQUENTIAL ? layered_seq_ops() : &OPS;
    m->layered = new (std::nothrow) CeraLayered();
    cera_hip_status st = m->layered ? CERA_HIP_OK : cera_fail(ctx, CERA_HIP_ERR_OOM, "host allocation failed");
    if (st == CERA_HIP_OK) {
        m->layered->cfg = *cfg;
        st = build(m, *cfg, layers);
    }
    if (st != CERA_HIP_OK) {
        const std::string keep = ctx->err;
        layered_destroy(m);
        ctx->err = keep;
        return st;
    }
    // the host pointers were borrowed for the call
    cera_hip_layered_config& c = m->layered->cfg;
    c.embed.data = c.pos.data = c.head.data = c.loop_in.data = nullptr;
    c.loop_step = c.final_norm = nullptr;
    m->cfg.n_layers = static_cast<uint32_t>(m->layered->runs.size() + m->layered->seq.size());
    m->cfg.hidden = cfg->width;
    m->cfg.vocab = cfg->vocab;
    m->cfg.max_seq_len = cfg->max_seq_len;
    *out = m;
    return CERA_HIP_OK;
}
