// What the readers of the layered architectures (nafevik.cpp, fidinex.cpp) share: access to config.json and to the
// tensors with the path of a key or the name of a tensor in every message, and what a reader fills in.
#pragma once
#include <cmath>
#include <cstring>
#include <memory>
#include <string>
#include <vector>

#include "cera_hip.h"
#include "hip_layered.h"
#include "safetensors.h"

namespace cera {

namespace layered {

[[noreturn]] inline void bail(const std::string& m) { throw BackendError(m); }

// config access with the path of a key in every message
struct ConfigNode {
    const Json* j;
    std::string path;
    bool has(const char* key) const {
        const Json* v = j->find(key);
        return v && !v->is_null();
    }
    ConfigNode at(const char* key) const {
        if (!has(key)) bail("config.json: missing " + path + key);
        return {j->find(key), path + key + "."};
    }
    std::string name() const { return path.substr(0, path.size() - 1); }
    double num() const {
        if (j->type != Json::Number || !std::isfinite(j->num)) bail("config.json: " + name() + " must be a number");
        return j->num;
    }
    uint32_t u32(uint32_t lo = 1) const {
        if (j->type != Json::Number || !j->is_int || j->integer < lo || j->integer > 0x7FFFFFFF)
            bail("config.json: " + name() + " must be an integer of at least " + std::to_string(lo));
        return static_cast<uint32_t>(j->integer);
    }
    bool flag() const {
        if (j->type != Json::Bool) bail("config.json: " + name() + " must be true or false");
        return j->b;
    }
    const std::string& str() const {
        if (j->type != Json::String) bail("config.json: " + name() + " must be a string");
        return j->str;
    }
};

struct LayeredWeights {
    std::unique_ptr<SafeTensors> file;
    std::vector<std::unique_ptr<std::vector<float>>> vectors;   // alive until the model is built

    const SafeTensor& get(const std::string& name, const std::vector<uint64_t>& shape) const {
        const SafeTensor* t = file->find(name);
        if (!t) bail("tensor " + name + " is missing");
        auto text = [](const std::vector<uint64_t>& s) {
            std::string o = "[";
            for (size_t i = 0; i < s.size(); ++i) o += (i ? ", " : "") + std::to_string(s[i]);
            return o + "]";
        };
        if (t->shape != shape) bail("tensor " + name + " has shape " + text(t->shape) + ", expected " + text(shape));
        if (t->dtype != "BF16") bail("tensor " + name + " is " + t->dtype + ", expected BF16");
        return *t;
    }
    cera_hip_tensor mat(const std::string& name, uint64_t m, uint64_t k) const {
        const SafeTensor& t = get(name, {m, k});
        cera_hip_tensor o{};
        o.ggml_type = CERA_HIP_BF16;
        o.m = m; o.k = k; o.data = t.data; o.nbytes = t.nbytes;
        return o;
    }
    // bf16 widened exactly
    const float* vec(const std::string& name, const std::vector<uint64_t>& shape) {
        const SafeTensor& t = get(name, shape);
        auto v = std::make_unique<std::vector<float>>(t.elements());
        for (size_t i = 0; i < v->size(); ++i) {
            uint16_t b;
            std::memcpy(&b, static_cast<const char*>(t.data) + 2 * i, 2);
            const uint32_t w = static_cast<uint32_t>(b) << 16;
            std::memcpy(&(*v)[i], &w, 4);
        }
        vectors.push_back(std::move(v));
        return vectors.back()->data();
    }
    const float* keep(std::vector<float> v) {
        vectors.push_back(std::make_unique<std::vector<float>>(std::move(v)));
        return vectors.back()->data();
    }
    // several vectors back to back
    const float* join(std::initializer_list<const float*> parts, std::initializer_list<uint64_t> sizes) {
        std::vector<float> v;
        auto n = sizes.begin();
        for (const float* p : parts) v.insert(v.end(), p, p + *n++);
        return keep(std::move(v));
    }
};

// A model as cera_hip_layered_create takes it, and what its snapshots hold per layer run in execution order.
struct Description {
    LayeredWeights weights;
    cera_hip_layered_config config{};
    std::vector<cera_hip_layered_layer> layers;
    std::vector<HipLayeredModel::LayerState> state;
};

// The entry of config.json's list for layer i, and the prefix of its tensors.  `layers` and config.n_layers are set up
// by read_layers.
inline std::vector<ConfigNode> read_layers(const ConfigNode& top, Description& d) {
    const Json* list = top.at("layers").j;
    if (list->type != Json::Array || list->arr.empty()) bail("config.json: layers must be a list of layers");
    std::vector<ConfigNode> nodes;
    for (size_t i = 0; i < list->arr.size(); ++i) nodes.push_back({&list->arr[i], "layers[" + std::to_string(i) + "]."});
    d.config.n_layers = static_cast<uint32_t>(nodes.size());
    d.layers.assign(nodes.size(), cera_hip_layered_layer{});
    return nodes;
}

// `context`: positions the caller asks for (SIZE_MAX: as many as there are)
void read_nafevik(const ConfigNode& top, size_t context, Description& d, ModelConfig& c);
void read_fidinex(const ConfigNode& top, size_t context, Description& d, ModelConfig& c);

}  // namespace layered
}  // namespace cera
