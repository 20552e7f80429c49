// HipLayeredModel: models described layer by layer in a config.json, with bfloat16 weights in a
// model.safetensors beside it, over cera_hip_layered_create.  One reader per architecture (layered_reader.h).
#pragma once
#include <memory>

#include "hip_device_model.h"
#include "load_model.h"

namespace cera {
namespace layered { struct Description; }

class HipLayeredModel final : public HipDeviceModel {
public:
    using HipDeviceModel::LayerState;
    // dir holds config.json (parsed: config) and model.safetensors.  Throw BackendError with the
    // reason on any failure.
    static std::unique_ptr<Model> nafevik(const std::string& dir, const Json& config, const LoadOptions& opt);
    static std::unique_ptr<Model> fidinex(const std::string& dir, const Json& config, const LoadOptions& opt);
    static std::unique_ptr<Model> create(const ModelConfig& c, const layered::Description& d, const LoadOptions& opt);

private:
    HipLayeredModel() = default;
    LayerState layer_state(size_t l) const override { return state_[l]; }
    std::vector<LayerState> state_;   // per layer run
};

}  // namespace cera
