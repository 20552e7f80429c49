// The `Model` trait as the backends here implement it, and the types that pass through it.
//
// Reference surface mirrored:
//   * trait Model                      cera/src/model/mod.rs:200-606
//   * forward_prefill_chunked default  cera/src/model/mod.rs:303-332
//
// Rust's forward methods are infallible by signature and the reference GPU
// backends panic on a device error; here such an error throws
// cera::BackendError, which the C face in hip_llama_capi.cpp turns into a
// status code so nothing unwinds across a C boundary.
#pragma once
#include <atomic>
#include <cstddef>
#include <cstdint>
#include <optional>
#include <stdexcept>
#include <string>
#include <utility>
#include <vector>

namespace cera {

struct BackendError : std::runtime_error {
    using std::runtime_error::runtime_error;
};

// cera/src/model/mod.rs:52-113
struct ScalarMultipliers {
    float embedding = 1.0f, residual = 1.0f;
    std::optional<float> attn;  // absent (or stored 0.0) => 1/sqrt(head_dim)
    float logit = 1.0f;
};

// cera/src/model/mod.rs:117-145 (the fields a dense transformer uses)
struct ModelConfig {
    std::string architecture;
    size_t n_layers = 0, hidden_size = 0, intermediate_size = 0, n_heads = 0, n_kv_heads = 0, head_dim = 0,
           vocab_size = 0, max_seq_len = 0;
    float rope_theta = 1000000.0f, rms_norm_eps = 1e-6f;
    ScalarMultipliers scalars;
};

// The KV cache lives in HBM inside the model; only the position counter is
// mirrored on the caller's side (InferenceState::seq_len in cera).
struct InferenceState {
    size_t seq_len = 0;
};

// cera/src/kv_cache.rs:1382-1396: per attention layer the raw f32 K and V bytes of rows
// [0, seq_len), time-major [pos][kv_dim] (LayerSnapshot::Attention).
// With an f16 cache the bytes are the raw little-endian half bits (LayerSnapshot::AttentionF16,
// cera/src/kv_cache.rs:1411-1421); `f16` is the variant tag restore checks.
struct LayerSnapshot {
    std::vector<uint8_t> k_data, v_data;
    bool f16 = false;
    // a layer with a short convolution (LayerSnapshot's convolution variant, cera/src/kv_cache.rs:1382-1421):
    // its last inputs, f32, oldest first
    std::vector<uint8_t> conv_data;
};
struct StateSnapshot {
    std::vector<LayerSnapshot> layers;
    size_t seq_len = 0;
};

// cera/src/kv_cache.rs:88-110, the modes a dense transformer on this backend honours
enum class KvCompression { None = 0, F16 = 1 };

// index of the largest value, the lowest one on ties (cera/src/sampler.rs:20-30)
uint32_t argmax_token(const std::vector<float>& logits);

// The subset of `trait Model` a text backend implements.
class Model {
public:
    virtual ~Model() = default;
    virtual std::vector<float> forward(const uint32_t* tokens, size_t n_tokens, size_t pos, InferenceState& state) = 0;
    virtual std::vector<float> forward_prefill(const uint32_t* tokens, size_t n_tokens, size_t start_pos,
                                               InferenceState& state);
    virtual uint32_t forward_greedy(const uint32_t* tokens, size_t n_tokens, size_t pos, InferenceState& state);
    // logits of every position, row-major [n_tokens * vocab]; empty unless supports_all_logits()
    virtual std::vector<float> forward_prefill_logits_all(const uint32_t*, size_t, size_t, InferenceState&) { return {}; }
    virtual void truncate_kv(InferenceState& state, size_t len) = 0;
    // n_keep context shift (cera/src/model/mod.rs:336-365): callers check supports_kv_shift() first
    virtual void shift_kv(InferenceState&, size_t /*n_keep*/, size_t /*shift*/) {}
    // prefix-cache snapshots (cera/src/model/mod.rs:507-533)
    virtual struct StateSnapshot snapshot_state();
    virtual void restore_state(const struct StateSnapshot&);
    // (tokens consumed, logits of the last processed chunk); chunks of `ubatch` (0 = one chunk),
    // `cancel` polled after each chunk.
    std::pair<size_t, std::optional<std::vector<float>>> forward_prefill_chunked(const uint32_t* tokens, size_t n_tokens,
                                                                                 size_t start_pos, InferenceState& state,
                                                                                 size_t ubatch,
                                                                                 const std::atomic<bool>& cancel);
    virtual const ModelConfig& config() const = 0;
    virtual uint64_t gpu_memory_bytes() const { return 0; }
    virtual bool supports_all_logits() const { return false; }
    virtual bool supports_kv_shift() const { return false; }
    virtual bool supports_embedding_input() const { return false; }
    virtual bool supports_hidden_states() const { return false; }
    virtual bool turboquant_supported() const { return false; }
    virtual bool f16_kv_supported() const { return false; }
    // cera/src/model/mod.rs:557-592: called before any forward pass; first call wins
    virtual void configure_kv_compression(KvCompression) {}
};

}  // namespace cera
