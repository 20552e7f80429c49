// The `Model` trait's defaults and HipDeviceModel over the C ABI of cera_hip.h.
#include "hip_device_model.h"

#include <algorithm>
#include <cmath>
#include <cstring>

#include "cera_host.h"

namespace cera {
namespace {

[[noreturn]] void bail(const std::string& m) { throw BackendError(m); }

}  // namespace

uint32_t argmax_token(const std::vector<float>& v) {
    uint32_t best = 0;
    float bv = -INFINITY;
    for (size_t i = 0; i < v.size(); ++i)
        if (v[i] > bv) { bv = v[i]; best = static_cast<uint32_t>(i); }
    return best;
}

// ---- trait defaults (cera/src/model/mod.rs:207-220, 303-332, 494-497) ----

std::vector<float> Model::forward_prefill(const uint32_t* tokens, size_t n, size_t start_pos, InferenceState& state) {
    std::vector<float> logits;
    for (size_t i = 0; i < n; ++i) logits = forward(tokens + i, 1, start_pos + i, state);
    return logits;
}

uint32_t Model::forward_greedy(const uint32_t* tokens, size_t n, size_t pos, InferenceState& state) {
    return argmax_token(forward(tokens, n, pos, state));
}

std::pair<size_t, std::optional<std::vector<float>>> Model::forward_prefill_chunked(
    const uint32_t* tokens, size_t n, size_t start_pos, InferenceState& state, size_t ubatch,
    const std::atomic<bool>& cancel) {
    if (ubatch == 0) ubatch = std::max<size_t>(n, 1);
    size_t consumed = 0;
    std::optional<std::vector<float>> last;
    while (consumed < n) {
        size_t len = std::min(ubatch, n - consumed);
        last = forward_prefill(tokens + consumed, len, start_pos + consumed, state);
        consumed += len;
        // polled after the chunk, so a cancel raised before the call still advances by one chunk
        if (cancel.load(std::memory_order_relaxed) && consumed < n) break;
    }
    return {consumed, std::move(last)};
}

// The trait defaults panic with unimplemented!(): a backend without device-resident state has
// nothing to snapshot (cera/src/model/mod.rs:521-533).
StateSnapshot Model::snapshot_state() { throw BackendError("snapshot_state not supported by this backend"); }
void Model::restore_state(const StateSnapshot&) { throw BackendError("restore_state not supported by this backend"); }

// ---- HipDeviceModel ----

HipDeviceModel::~HipDeviceModel() {
    if (model_) cera_hip_model_destroy(model_);
    if (ctx_) cera_hip_ctx_destroy(ctx_);
}

void HipDeviceModel::open_context(int device) {
    if (cera_hip_ctx_create(device, nullptr, &ctx_) != CERA_HIP_OK)
        bail(std::string("hip context: ") + cera_hip_last_error(nullptr));
}

void HipDeviceModel::device_panic(const char* what) const {
    throw BackendError(std::string(what) + ": " + cera_hip_last_error(ctx_));
}

std::vector<float> HipDeviceModel::forward(const uint32_t* tokens, size_t n, size_t pos, InferenceState& state) {
    if (n != 1) bail("forward expects single token");
    if (tokens[0] >= config_.vocab_size)
        bail("token_id " + std::to_string(tokens[0]) + " out of range (vocab_size=" + std::to_string(config_.vocab_size) + ")");
    std::vector<float> logits(config_.vocab_size);
    if (cera_hip_forward(model_, tokens[0], static_cast<uint32_t>(pos), logits.data()) != CERA_HIP_OK)
        device_panic("forward");
    state.seq_len = cera_hip_seq_len(model_);
    return logits;
}

std::vector<float> HipDeviceModel::forward_prefill(const uint32_t* tokens, size_t n, size_t start_pos,
                                                  InferenceState& state) {
    if (n == 0) bail("forward_prefill requires at least one token");
    if (start_pos != state.seq_len)
        bail("forward_prefill: start_pos (" + std::to_string(start_pos) + ") must equal state.seq_len (" +
             std::to_string(state.seq_len) + ")");
    std::vector<float> logits(config_.vocab_size);
    if (cera_hip_forward_prefill(model_, tokens, static_cast<uint32_t>(n), static_cast<uint32_t>(start_pos),
                                 logits.data()) != CERA_HIP_OK)
        device_panic("forward_prefill");
    state.seq_len = cera_hip_seq_len(model_);
    return logits;
}

std::vector<float> HipDeviceModel::forward_prefill_logits_all(const uint32_t* tokens, size_t n, size_t start_pos,
                                                             InferenceState& state) {
    if (n == 0) bail("forward_prefill_logits_all requires at least one token");
    if (start_pos != state.seq_len)
        bail("forward_prefill_logits_all: start_pos (" + std::to_string(start_pos) + ") must equal state.seq_len (" +
             std::to_string(state.seq_len) + ")");
    std::vector<float> logits(n * config_.vocab_size);
    if (cera_hip_forward_prefill_logits_all(model_, tokens, static_cast<uint32_t>(n), static_cast<uint32_t>(start_pos),
                                            logits.data()) != CERA_HIP_OK)
        device_panic("forward_prefill_logits_all");
    state.seq_len = cera_hip_seq_len(model_);
    return logits;
}

uint32_t HipDeviceModel::forward_greedy(const uint32_t* tokens, size_t n, size_t pos, InferenceState& state) {
    if (n != 1) bail("forward_greedy expects single token");
    uint32_t next = 0;
    if (cera_hip_forward_greedy(model_, tokens[0], static_cast<uint32_t>(pos), &next) != CERA_HIP_OK)
        device_panic("forward_greedy");
    state.seq_len = cera_hip_seq_len(model_);
    return next;
}

void HipDeviceModel::truncate_kv(InferenceState& state, size_t len) {
    if (len > state.seq_len)
        bail("truncate_kv: len (" + std::to_string(len) + ") exceeds seq_len (" + std::to_string(state.seq_len) + ")");
    if (cera_hip_truncate_kv(model_, static_cast<uint32_t>(len)) != CERA_HIP_OK) device_panic("truncate_kv");
    state.seq_len = len;
}

// the integer-only converters of the host library (the reference's, cera/src/quant.rs:48-164)
static uint16_t half_bits(float v) { return cera_f32_to_f16(v); }
static float half_value(uint16_t b) { return cera_f16_to_f32(b); }

namespace {
// f32 values as the bytes a snapshot holds: raw f32, or the half bits of an f16 cache (read_kv widened
// them exactly, so narrowing gives them back)
std::vector<uint8_t> pack(const std::vector<float>& v, bool f16) {
    std::vector<uint8_t> out(v.size() * (f16 ? 2 : 4));
    if (!f16) {
        if (!v.empty()) std::memcpy(out.data(), v.data(), out.size());
        return out;
    }
    for (size_t i = 0; i < v.size(); ++i) {
        const uint16_t b = half_bits(v[i]);
        std::memcpy(out.data() + 2 * i, &b, 2);
    }
    return out;
}
std::vector<float> unpack(const std::vector<uint8_t>& b, bool f16) {
    std::vector<float> out(b.size() / (f16 ? 2 : 4));
    if (!f16) {
        if (!out.empty()) std::memcpy(out.data(), b.data(), b.size());
        return out;
    }
    for (size_t i = 0; i < out.size(); ++i) {
        uint16_t h;
        std::memcpy(&h, b.data() + 2 * i, 2);
        out[i] = half_value(h);
    }
    return out;
}
}  // namespace

StateSnapshot HipDeviceModel::snapshot_state() {
    StateSnapshot snap;
    snap.seq_len = cera_hip_seq_len(model_);
    const bool f16 = kv_compression() == KvCompression::F16;
    snap.layers.resize(state_layers());
    for (size_t l = 0; l < snap.layers.size(); ++l) {
        const LayerState ls = layer_state(l);
        LayerSnapshot& L = snap.layers[l];
        L.f16 = f16;
        std::vector<float> k(snap.seq_len * ls.k), v(snap.seq_len * ls.v), conv(ls.conv);
        if (snap.seq_len && cera_hip_read_kv(model_, static_cast<uint32_t>(l), k.data(), v.data()) != CERA_HIP_OK)
            device_panic("snapshot_state");
        if (ls.conv && cera_hip_read_conv(model_, static_cast<uint32_t>(l), conv.data()) != CERA_HIP_OK) device_panic("snapshot_state");
        L.k_data = pack(k, f16);
        L.v_data = pack(v, f16);
        L.conv_data = pack(conv, false);
    }
    return snap;
}

void HipDeviceModel::restore_state(const StateSnapshot& snap) {
    const bool f16 = kv_compression() == KvCompression::F16;
    const size_t esz = f16 ? 2 : 4;
    if (snap.layers.size() != state_layers()) bail("restore_state: snapshot has " + std::to_string(snap.layers.size()) +
                                                   " layers, model has " + std::to_string(state_layers()));
    if (snap.seq_len > config_.max_seq_len) bail("restore_state: snapshot is longer than the context");
    for (size_t l = 0; l < snap.layers.size(); ++l) {
        const LayerSnapshot& L = snap.layers[l];
        const LayerState ls = layer_state(l);
        // the cross-mode gate: an f16 snapshot never loads into an f32 cache or the reverse
        if (L.f16 != f16) bail("restore_state: snapshot and model disagree on the KV cache element type");
        if (L.k_data.size() != snap.seq_len * ls.k * esz || L.v_data.size() != snap.seq_len * ls.v * esz || L.conv_data.size() != ls.conv * 4)
            bail("restore_state: layer byte length does not match seq_len * kv_dim * element size");
    }
    for (size_t l = 0; l < snap.layers.size(); ++l) {
        const LayerSnapshot& L = snap.layers[l];
        const std::vector<float> k = unpack(L.k_data, f16), v = unpack(L.v_data, f16), conv = unpack(L.conv_data, false);
        const uint32_t n = static_cast<uint32_t>(snap.seq_len);
        if (cera_hip_write_kv(model_, static_cast<uint32_t>(l), k.data(), v.data(), n) != CERA_HIP_OK) device_panic("restore_state");
        if (!conv.empty() && cera_hip_write_conv(model_, static_cast<uint32_t>(l), conv.data(), n) != CERA_HIP_OK) device_panic("restore_state");
    }
    if (cera_hip_set_seq_len(model_, static_cast<uint32_t>(snap.seq_len)) != CERA_HIP_OK) device_panic("restore_state");
}

uint64_t HipDeviceModel::gpu_memory_bytes() const { return cera_hip_memory_bytes(model_); }

std::string HipDeviceModel::device_name() const {
    char name[256] = {0};
    uint32_t cu = 0;
    uint64_t hbm = 0;
    if (cera_hip_device_info(ctx_, name, &cu, &hbm) != CERA_HIP_OK) return "unknown";
    return std::string(name) + " (" + std::to_string(cu) + " CUs, " + std::to_string(hbm >> 30) + " GiB)";
}

}  // namespace cera
