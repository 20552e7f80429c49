// HipLayeredModel: models described layer by layer in a config.json, with bfloat16 weights in a
// model.safetensors beside it, over cera_hip_layered_create.
//
// Architectures: "Nafevik" -- embedding plus learned positions; parallel attention and gated
// feed-forward behind one RMS norm, each reading its input through a short causal convolution; sigmoid
// attention inside chunks, with YaRN rotation in adjacent pairs and a gate per head; a range of
// layers run several times, each pass starting from a product over the residual and the embedding.
#pragma once
#include <memory>

#include "hip_device_model.h"
#include "load_model.h"

namespace cera {

class HipLayeredModel final : public HipDeviceModel {
public:
    // dir holds config.json (parsed: config) and model.safetensors.  Throws BackendError with the
    // reason on any failure.
    static std::unique_ptr<Model> from_dir(const std::string& dir, const Json& config, const LoadOptions& opt);

private:
    HipLayeredModel() = default;
    LayerState layer_state(size_t l) const override { return state_[l]; }
    std::vector<LayerState> state_;   // per layer run
};

}  // namespace cera
