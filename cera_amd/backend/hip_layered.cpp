// HipLayeredModel: a model directory through its architecture's reader -> cera_hip_layered_create.
#include "layered_reader.h"

namespace cera {
namespace {

using layered::bail;

std::unique_ptr<Model> load(const std::string& dir, const Json& config, const LoadOptions& opt,
                            void (*read)(const layered::ConfigNode&, size_t, layered::Description&, ModelConfig&)) {
    if (opt.context_size == 0) bail("context_size must be > 0");
    const layered::ConfigNode top{&config, ""};
    std::string err;
    layered::Description d;
    d.weights.file = SafeTensors::open(dir + "/model.safetensors", &err);
    if (!d.weights.file) bail(err);
    ModelConfig c;
    c.architecture = top.at("architecture").str();
    d.config.f32 = opt.f32 ? 1 : 0;
    read(top, opt.context_size, d, c);
    return HipLayeredModel::create(c, d, opt);
}

}  // namespace

std::unique_ptr<Model> HipLayeredModel::nafevik(const std::string& dir, const Json& config, const LoadOptions& opt) {
    return load(dir, config, opt, layered::read_nafevik);
}
std::unique_ptr<Model> HipLayeredModel::fidinex(const std::string& dir, const Json& config, const LoadOptions& opt) {
    return load(dir, config, opt, layered::read_fidinex);
}

std::unique_ptr<Model> HipLayeredModel::create(const ModelConfig& c, const layered::Description& d, const LoadOptions& opt) {
    std::unique_ptr<HipLayeredModel> self(new HipLayeredModel());
    self->config_ = c;
    self->state_ = d.state;
    self->open_context(opt.device);
    if (cera_hip_layered_create(self->ctx_, &d.config, d.layers.data(), &self->model_) != CERA_HIP_OK)
        bail(std::string("hip model: ") + cera_hip_last_error(self->ctx_));
    return self;
}

}  // namespace cera
