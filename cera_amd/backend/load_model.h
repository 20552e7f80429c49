// Model registry: which class loads a path.
//   * a directory with a config.json: by its "architecture" (load_model_dir)
//   * anything else: a GGUF file, by its general.architecture (load_model_hip)
#pragma once
#include <memory>
#include <string>

#include "json.h"
#include "model.h"

namespace cera {

class GgufFile;

struct LoadOptions {
    size_t context_size = 1024;
    int device = 0;
    bool f32 = false;   // run in f32 instead of bf16 (models with float weights)
};

// load_model_gpu's twin (cera/src/model/mod.rs:672-703): arch allow-list, then the model.
std::unique_ptr<Model> load_model_hip(const GgufFile& gguf, size_t context_size, int device = 0);
std::unique_ptr<Model> load_model_dir(const std::string& dir, const LoadOptions& opt);
bool is_model_dir(const std::string& path);
// any path; throws BackendError
std::unique_ptr<Model> load_model(const std::string& path, const LoadOptions& opt);

}  // namespace cera
