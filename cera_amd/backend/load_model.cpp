// Registry, the GGUF half and the entry for any path (load_model.h).
#include "load_model.h"

#include "gguf.h"
#include "hip_llama.h"

namespace cera {

std::unique_ptr<Model> load_model_hip(const GgufFile& gguf, size_t context_size, int device) {
    std::string arch = gguf.get_str("general.architecture").value_or("unknown");
    if (arch == "qwen2" || arch == "qwen3" || arch == "llama" || arch == "granite")
        return HipLlamaModel::from_gguf(gguf, context_size, device);
    throw BackendError("unsupported architecture for hip: " + arch);
}

std::unique_ptr<Model> load_model(const std::string& path, const LoadOptions& opt) {
    if (is_model_dir(path)) return load_model_dir(path, opt);
    if (opt.f32) throw BackendError("dtype f32 is for models with float weights; a GGUF file runs in its block types");
    std::string err;
    auto g = GgufFile::open(path, &err);
    if (!g) throw BackendError(err);
    return load_model_hip(*g, opt.context_size, opt.device);   // the weights are in HBM afterwards
}

}  // namespace cera
