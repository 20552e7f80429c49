// What every model family on the hip backend shares above the C ABI: the `Model` methods over a
// cera_hip_model handle, the device-resident-KV contract (cera/src/model/mod.rs:176-199, 251-283: the
// backend keeps its own position counter and keeps InferenceState::seq_len equal to it), snapshots.
#pragma once
#include "cera_hip.h"
#include "model.h"

namespace cera {

class HipDeviceModel : public Model {
public:
    ~HipDeviceModel() override;
    HipDeviceModel(const HipDeviceModel&) = delete;
    HipDeviceModel& operator=(const HipDeviceModel&) = delete;

    std::vector<float> forward(const uint32_t* tokens, size_t n_tokens, size_t pos, InferenceState& state) override;
    std::vector<float> forward_prefill(const uint32_t* tokens, size_t n_tokens, size_t start_pos,
                                       InferenceState& state) override;
    uint32_t forward_greedy(const uint32_t* tokens, size_t n_tokens, size_t pos, InferenceState& state) override;
    std::vector<float> forward_prefill_logits_all(const uint32_t* tokens, size_t n_tokens, size_t start_pos,
                                                  InferenceState& state) override;
    bool supports_all_logits() const override { return true; }
    void truncate_kv(InferenceState& state, size_t len) override;
    StateSnapshot snapshot_state() override;
    void restore_state(const StateSnapshot& snapshot) override;
    const ModelConfig& config() const override { return config_; }
    uint64_t gpu_memory_bytes() const override;
    virtual KvCompression kv_compression() const { return KvCompression::None; }
    std::string device_name() const;
    // floats of one cached K row / V row / the convolution state of a layer (0: none)
    struct LayerState { size_t k = 0, v = 0, conv = 0; };

protected:
    HipDeviceModel() = default;
    [[noreturn]] void device_panic(const char* what) const;
    void open_context(int device);
    virtual LayerState layer_state(size_t l) const = 0;
    virtual size_t state_layers() const { return config_.n_layers; }

    ModelConfig config_;
    cera_hip_ctx* ctx_ = nullptr;
    cera_hip_model* model_ = nullptr;
};

}  // namespace cera
