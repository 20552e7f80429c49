// Registry of the models that come as a directory (load_model.h).
#include <sys/stat.h>

#include <fstream>
#include <sstream>

#include "hip_layered.h"
#include "load_model.h"

namespace cera {
namespace {

struct DirModel {
    const char* architecture;
    std::unique_ptr<Model> (*load)(const std::string& dir, const Json& config, const LoadOptions& opt);
};
const DirModel MODELS[] = {
    {"Nafevik", HipLayeredModel::nafevik},
    {"Fidinex", HipLayeredModel::fidinex},
};

}  // namespace

bool is_model_dir(const std::string& path) {
    struct stat st;
    return stat(path.c_str(), &st) == 0 && S_ISDIR(st.st_mode);
}

std::unique_ptr<Model> load_model_dir(const std::string& dir, const LoadOptions& opt) {
    std::ifstream f(dir + "/config.json", std::ios::binary);
    if (!f) throw BackendError(dir + "/config.json cannot be read");
    std::stringstream text;
    text << f.rdbuf();
    Json config;
    std::string err;
    if (!Json::parse(text.str(), &config, &err)) throw BackendError(dir + "/config.json: " + err);
    const Json* arch = config.find("architecture");
    if (!arch || arch->type != Json::String) throw BackendError(dir + "/config.json: missing architecture");
    for (const DirModel& m : MODELS)
        if (arch->str == m.architecture) return m.load(dir, config, opt);
    throw BackendError("unsupported architecture for hip: " + arch->str);
}

}  // namespace cera
