// C ABI, model level: the calls every model family answers -- forward / forward_greedy /
// forward_prefill / truncate_kv / snapshots (the `Model` trait, cera/src/model/mod.rs:200-606) --
// with the argument checks, the position counter and the locking in one place.  What a family does
// for a call is in its CeraModelOps (model.h).
#include <algorithm>
#include <cstring>

#include "glue.hip.h"
#include "model.h"

cera_hip_status cera_pinned_word(cera_hip_ctx* ctx, uint32_t** host, uint32_t** dev) {
    if (!ctx->word_host) {
        void *h = nullptr, *d = nullptr;
        HIP_TRY(ctx, hipHostMalloc(&h, 64, hipHostMallocMapped));
        const hipError_t e = hipHostGetDevicePointer(&d, h, 0);
        if (e != hipSuccess) {
            (void)hipHostFree(h);
            return cera_fail(ctx, CERA_HIP_ERR_DEVICE, std::string("hipHostGetDevicePointer: ") + hipGetErrorString(e));
        }
        ctx->word_host = static_cast<uint32_t*>(h);
        ctx->word_dev = static_cast<uint32_t*>(d);
    }
    *host = ctx->word_host;
    *dev = ctx->word_dev;
    return CERA_HIP_OK;
}

cera_hip_status cera_launch_argmax(cera_hip_ctx* ctx, const float* x, uint32_t n, uint32_t* out_dev, uint32_t* out_host_mapped) {
    void* part;
    CERA_TRY(cera_scratch(ctx, 8, ARGMAX_PARTS * 8, &part));
    float* pv = static_cast<float*>(part);
    uint32_t* pi = reinterpret_cast<uint32_t*>(pv + ARGMAX_PARTS);
    const uint32_t np = std::max(1u, std::min<uint32_t>(ARGMAX_PARTS, (n + 1023) / 1024));
    hipLaunchKernelGGL(argmax_partial_kernel, dim3(np), dim3(256), 0, ctx->stream, x, n, pv, pi);
    hipLaunchKernelGGL(argmax_final_kernel, dim3(1), dim3(256), 0, ctx->stream, pv, pi, np, out_dev, out_host_mapped);
    HIP_TRY(ctx, hipGetLastError());
    return CERA_HIP_OK;
}

// ---------------------------------------------------------------------------
extern "C" void cera_hip_model_destroy(cera_hip_model* m) {
    if (m) m->ops->destroy(m);
}
extern "C" uint32_t cera_hip_seq_len(const cera_hip_model* m) { return m ? m->seq_len : 0; }
extern "C" uint64_t cera_hip_memory_bytes(const cera_hip_model* m) { return m ? m->bytes : 0; }

extern "C" cera_hip_status cera_hip_truncate_kv(cera_hip_model* m, uint32_t len) {
    if (!m) return CERA_HIP_ERR_ARGUMENT;
    ModelLock lk(m);
    if (len >= m->seq_len) return CERA_HIP_OK;
    if (m->ops->truncate) CERA_TRY(m->ops->truncate(m, len));
    m->seq_len = len;  // rows past len are simply overwritten later
    return CERA_HIP_OK;
}

extern "C" cera_hip_status cera_hip_set_seq_len(cera_hip_model* m, uint32_t len) {
    if (!m) return CERA_HIP_ERR_ARGUMENT;
    ModelLock lk(m);
    if (len > m->cfg.max_seq_len) return cera_fail(m->ctx, CERA_HIP_ERR_POSITION, "set_seq_len: beyond max_seq_len");
    m->seq_len = len;
    return CERA_HIP_OK;
}

// Prefix-cache snapshots (Model::snapshot_state / restore_state, cera/src/model/mod.rs:507-533;
// layer layout LayerSnapshot::Attention, cera/src/kv_cache.rs:1382-1396): a layer's K and V as
// time-major [n_pos][kv_dim] f32, the CPU state's own layout.  cera_hip_read_kv is the snapshot
// side, cera_hip_write_kv the restore side: call it for every layer, then cera_hip_set_seq_len.
extern "C" cera_hip_status cera_hip_write_kv(cera_hip_model* m, uint32_t layer, const float* k, const float* v,
                                             uint32_t n_pos) {
    if (!m || (n_pos && (!k || !v)) || layer >= m->cfg.n_layers) return CERA_HIP_ERR_ARGUMENT;
    ModelLock lk(m);
    if (n_pos > m->cfg.max_seq_len) return cera_fail(m->ctx, CERA_HIP_ERR_POSITION, "write_kv: more positions than max_seq_len");
    return m->ops->write_kv(m, layer, k, v, n_pos);
}

extern "C" cera_hip_status cera_hip_read_kv(cera_hip_model* m, uint32_t layer, float* k_out, float* v_out) {
    if (!m || !k_out || !v_out || layer >= m->cfg.n_layers) return CERA_HIP_ERR_ARGUMENT;
    ModelLock lk(m);
    return m->ops->read_kv(m, layer, k_out, v_out);
}

// The convolution half of a snapshot (LayerSnapshot's short-convolution variant,
// cera/src/kv_cache.rs:1382-1421): nothing to do for a family without one.
extern "C" cera_hip_status cera_hip_read_conv(cera_hip_model* m, uint32_t layer, float* rows) {
    if (!m || !rows || layer >= m->cfg.n_layers) return CERA_HIP_ERR_ARGUMENT;
    ModelLock lk(m);
    return m->ops->read_conv ? m->ops->read_conv(m, layer, rows) : CERA_HIP_OK;
}
extern "C" cera_hip_status cera_hip_write_conv(cera_hip_model* m, uint32_t layer, const float* rows, uint32_t n_pos) {
    if (!m || !rows || layer >= m->cfg.n_layers) return CERA_HIP_ERR_ARGUMENT;
    ModelLock lk(m);
    if (n_pos > m->cfg.max_seq_len) return cera_fail(m->ctx, CERA_HIP_ERR_POSITION, "write_conv: more positions than max_seq_len");
    return m->ops->write_conv ? m->ops->write_conv(m, layer, rows, n_pos) : CERA_HIP_OK;
}

// A call at position 0 starts a fresh sequence: callers hand a new InferenceState to every
// generate(), and a device-resident backend resets its own counter then, as the reference's do
// (cera/src/model/metal_lfm2.rs:4091-4096, gpu_lfm2.rs:3755-3762).  Cached rows are simply
// overwritten.
static cera_hip_status begin_at(cera_hip_model* m, uint32_t pos) {
    if (m->kv_broken) return cera_fail(m->ctx, CERA_HIP_ERR_DEVICE, "the model's KV cache is unusable (a cache re-allocation failed)");
    if (pos == 0) m->seq_len = 0;
    return CERA_HIP_OK;
}

static cera_hip_status check_step(cera_hip_model* m, uint32_t token, uint32_t pos) {
    CERA_TRY(begin_at(m, pos));
    if (token >= m->cfg.vocab)
        return cera_fail(m->ctx, CERA_HIP_ERR_ARGUMENT, "token id " + std::to_string(token) + " out of range (vocab " + std::to_string(m->cfg.vocab) + ")");
    if (pos != m->seq_len)
        return cera_fail(m->ctx, CERA_HIP_ERR_POSITION, "pos " + std::to_string(pos) + " != seq_len " + std::to_string(m->seq_len));
    if (pos >= m->cfg.max_seq_len)
        return cera_fail(m->ctx, CERA_HIP_ERR_POSITION, "context full: pos " + std::to_string(pos) + " >= max_seq_len " + std::to_string(m->cfg.max_seq_len));
    return CERA_HIP_OK;
}

extern "C" cera_hip_status cera_hip_forward(cera_hip_model* m, uint32_t token, uint32_t pos, float* logits) {
    if (!m || !logits) return CERA_HIP_ERR_ARGUMENT;
    ModelLock lk(m);
    CERA_TRY(check_step(m, token, pos));
    CERA_TRY(m->ops->decode(m, token, pos, true));
    CERA_TRY(cera_hip_download(m->ctx, logits, m->logits, static_cast<uint64_t>(m->cfg.vocab) * 4));
    m->seq_len = pos + 1;
    return CERA_HIP_OK;
}

extern "C" cera_hip_status cera_hip_forward_greedy(cera_hip_model* m, uint32_t token, uint32_t pos, uint32_t* next) {
    if (!m || !next) return CERA_HIP_ERR_ARGUMENT;
    ModelLock lk(m);
    CERA_TRY(check_step(m, token, pos));
    CERA_TRY(m->ops->decode(m, token, pos, true));
    // the argmax kernel writes the token into pinned host memory itself: no copy launch behind it
    uint32_t *word_host, *word_dev;
    CERA_TRY(cera_pinned_word(m->ctx, &word_host, &word_dev));
    CERA_TRY(cera_launch_argmax(m->ctx, m->logits, m->cfg.vocab, m->scalars + 2, word_dev));
    HIP_TRY(m->ctx, hipStreamSynchronize(m->ctx->stream));
    *next = *static_cast<volatile uint32_t*>(word_host);
    m->seq_len = pos + 1;
    return CERA_HIP_OK;
}

extern "C" cera_hip_status cera_hip_forward_prefill(cera_hip_model* m, const uint32_t* tokens, uint32_t n,
                                                    uint32_t start_pos, float* last_logits) {
    if (!m || !tokens || !last_logits) return CERA_HIP_ERR_ARGUMENT;
    if (n == 0) return cera_fail(m->ctx, CERA_HIP_ERR_ARGUMENT, "forward_prefill requires at least one token");
    ModelLock lk(m);
    CERA_TRY(begin_at(m, start_pos));
    if (start_pos != m->seq_len)
        return cera_fail(m->ctx, CERA_HIP_ERR_POSITION, "forward_prefill: start_pos " + std::to_string(start_pos) +
                                                            " must equal seq_len " + std::to_string(m->seq_len));
    if (static_cast<uint64_t>(start_pos) + n > m->cfg.max_seq_len)
        return cera_fail(m->ctx, CERA_HIP_ERR_POSITION, "forward_prefill: prompt does not fit max_seq_len");
    for (uint32_t i = 0; i < n; ++i)
        if (tokens[i] >= m->cfg.vocab) return cera_fail(m->ctx, CERA_HIP_ERR_ARGUMENT, "token id out of range");
    return m->ops->prefill(m, tokens, n, start_pos, last_logits);
}

extern "C" cera_hip_status cera_hip_forward_prefill_logits_all(cera_hip_model* m, const uint32_t* tokens, uint32_t n,
                                                               uint32_t start_pos, float* logits_all) {
    if (!m || !tokens || !logits_all) return CERA_HIP_ERR_ARGUMENT;
    if (n == 0) return cera_fail(m->ctx, CERA_HIP_ERR_ARGUMENT, "forward_prefill_logits_all requires at least one token");
    ModelLock lk(m);
    CERA_TRY(begin_at(m, start_pos));
    if (start_pos != m->seq_len)
        return cera_fail(m->ctx, CERA_HIP_ERR_POSITION, "forward_prefill_logits_all: start_pos " + std::to_string(start_pos) +
                                                            " must equal seq_len " + std::to_string(m->seq_len));
    if (static_cast<uint64_t>(start_pos) + n > m->cfg.max_seq_len)
        return cera_fail(m->ctx, CERA_HIP_ERR_POSITION, "forward_prefill_logits_all: tokens do not fit max_seq_len");
    for (uint32_t i = 0; i < n; ++i)
        if (tokens[i] >= m->cfg.vocab) return cera_fail(m->ctx, CERA_HIP_ERR_ARGUMENT, "token id out of range");
    return m->ops->prefill_all(m, tokens, n, start_pos, logits_all);
}

extern "C" cera_hip_status cera_hip_read_hidden(cera_hip_model* m, float* hidden_out) {
    if (!m || !hidden_out) return CERA_HIP_ERR_ARGUMENT;
    ModelLock lk(m);
    return cera_hip_download(m->ctx, hidden_out, m->hidden, static_cast<uint64_t>(m->cfg.hidden) * 4);
}

