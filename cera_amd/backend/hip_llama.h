// HipLlamaModel: the `Model`-trait implementation a `--device hip` backend adds
// to cera, written against the C-ABI of cera_hip.h only (the same calls a Rust
// `impl Model for HipLlamaModel` over a -sys crate would make).
//
// Reference surface mirrored here:
//   * LlamaModel::from_gguf_with_id    cera/src/model/llama.rs:158-450 (metadata keys, defaults,
//                                      load-time checks, optional tensors)
#pragma once
#include <memory>

#include "gguf.h"
#include "hip_device_model.h"

namespace cera {

enum class RopeType { Neox = 0, Norm = 1 };

class HipLlamaModel final : public HipDeviceModel {
public:
    // Parses metadata, resolves every tensor in the mapping and uploads it to HBM in
    // its native block layout.  Throws BackendError with the reason on any failure
    // (missing key/tensor, unsupported arch or tensor type, shape mismatch, device error).
    static std::unique_ptr<HipLlamaModel> from_gguf(const GgufFile& gguf, size_t context_size, int device = 0);
    // the shift kernel is instantiated for the head sizes models use
    bool supports_kv_shift() const override {
        const size_t hd = config_.head_dim;
        return hd == 32 || hd == 64 || hd == 80 || hd == 96 || hd == 128 || hd == 256;
    }
    bool f16_kv_supported() const override { return true; }
    void configure_kv_compression(KvCompression mode) override;
    KvCompression kv_compression() const override;
    void shift_kv(InferenceState& state, size_t n_keep, size_t shift) override;

    // verification hook: run every forward on the reference-order kernels (bit-identical to the
    // CPU AVX2 path, many times slower); only with an empty cache
    // 0 off, 1 reference order with per-token prefill, 2 with the x86 host's batched prefill (cera_hip.h)
    void set_reference_order(uint32_t mode);
    RopeType rope_type() const { return rope_type_; }

private:
    HipLlamaModel() = default;
    LayerState layer_state(size_t) const override {
        const size_t row = config_.n_kv_heads * config_.head_dim;
        return {row, row, 0};
    }
    RopeType rope_type_ = RopeType::Norm;
};

}  // namespace cera
