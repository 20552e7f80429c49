// HipLayeredModel: config.json and tensor names -> cera_hip_layered_create.
#include "hip_layered.h"

#include <algorithm>
#include <cmath>
#include <cstring>

#include "safetensors.h"

namespace cera {
namespace {

[[noreturn]] void bail(const std::string& m) { throw BackendError(m); }

// config access with the path of a key in every message
struct Node {
    const Json* j;
    std::string path;
    bool has(const char* key) const {
        const Json* v = j->find(key);
        return v && !v->is_null();
    }
    Node at(const char* key) const {
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
    const std::string& str() const {
        if (j->type != Json::String) bail("config.json: " + name() + " must be a string");
        return j->str;
    }
};

struct Weights {
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
};

cera_hip_attn_spec read_attention(const Node& m) {
    cera_hip_attn_spec a{};
    a.heads = m.at("heads").u32();
    a.kv_heads = m.at("kv_heads").u32();
    a.dim = m.at("dim").u32();
    a.vdim = m.at("vdim").u32();
    a.scale = static_cast<float>(m.at("scale").num());
    if (m.has("mask")) a.chunk = m.at("mask").at("size").u32();
    if (m.has("rot")) {
        const Node r = m.at("rot");
        a.rot_dims = r.at("dims").u32(0);
        a.rot_base = r.at("base").num();
        if (r.has("scaling")) {
            const Node s = r.at("scaling");
            a.yarn = 1;
            a.yarn_factor = s.at("factor").num();
            a.yarn_original = s.at("original").num();
            a.yarn_fast = s.at("fast").num();
            a.yarn_slow = s.at("slow").num();
        }
    }
    return a;
}

}  // namespace

std::unique_ptr<Model> HipLayeredModel::from_dir(const std::string& dir, const Json& config, const LoadOptions& opt) {
    if (opt.context_size == 0) bail("context_size must be > 0");
    const Node top{&config, ""};
    std::string err;
    Weights w;
    w.file = SafeTensors::open(dir + "/model.safetensors", &err);
    if (!w.file) bail(err);

    std::unique_ptr<HipLayeredModel> self(new HipLayeredModel());
    ModelConfig& c = self->config_;
    cera_hip_layered_config hc{};
    c.architecture = top.at("architecture").str();
    hc.width = top.at("width").u32();
    hc.vocab = top.at("vocab").u32();
    hc.conv_taps = top.at("canon").at("taps").u32();
    hc.eps = static_cast<float>(top.at("norm").at("eps").num());
    hc.residual_mult = static_cast<float>(top.at("residual_mult").num());
    hc.f32 = opt.f32 ? 1 : 0;
    const uint32_t positions = top.at("max_positions").u32();
    hc.max_seq_len = static_cast<uint32_t>(std::min<size_t>(opt.context_size, positions));
    const Json* list = top.at("layers").j;
    if (list->type != Json::Array || list->arr.empty()) bail("config.json: layers must be a list of layers");
    hc.n_layers = static_cast<uint32_t>(list->arr.size());
    const uint64_t width = hc.width;
    hc.embed = w.mat("embed", hc.vocab, width);
    hc.pos = w.mat("pos", positions, width);
    hc.head = w.mat("head", hc.vocab, width);
    hc.final_norm = w.vec("final.norm", {width});
    if (top.has("loop")) {
        const Node l = top.at("loop");
        hc.loop_start = l.at("start").u32(0);
        hc.loop_stop = l.at("stop").u32();
        hc.loop_times = l.at("times").u32();
        if (hc.loop_start >= hc.loop_stop || hc.loop_stop > hc.n_layers) bail("config.json: loop.start / loop.stop are no range of layers");
        hc.loop_in = w.mat("loop.in", width, 2 * width);
        hc.loop_step = w.vec("loop.step", {hc.loop_times, width});
    }

    std::vector<cera_hip_layered_layer> layers(hc.n_layers);
    for (uint32_t i = 0; i < hc.n_layers; ++i) {
        const Node l{&list->arr[i], "layers[" + std::to_string(i) + "]."};
        const std::string p = "l" + std::to_string(i) + ".";
        cera_hip_layered_layer& Y = layers[i];
        std::memset(&Y, 0, sizeof Y);
        const std::string& type = l.at("type").str();
        if (type != "attention") bail("config.json: " + l.path + "type: no mixer " + type);
        Y.attn = read_attention(l.at("mixer"));
        const cera_hip_attn_spec& a = Y.attn;
        const uint64_t H = a.heads, G = a.kv_heads;
        Y.norm = w.vec(p + "norm1", {width});
        Y.conv_attn = w.vec(p + "canon1", {width, hc.conv_taps});
        Y.score_bias = w.vec(p + "mix.pb", {H});
        Y.q = w.mat(p + "mix.q", H * a.dim, width);
        Y.k = w.mat(p + "mix.k", G * a.dim, width);
        Y.v = w.mat(p + "mix.v", G * a.vdim, width);
        Y.head_gate = w.mat(p + "mix.g", H, width);
        Y.o = w.mat(p + "mix.o", width, H * a.vdim);
        if (l.has("mlp")) {
            const Node f = l.at("mlp");
            if (f.at("kind").str() != "dense") bail("config.json: " + f.path + "kind: no feed-forward " + f.at("kind").str());
            Y.ff = f.at("ff").u32();
            Y.conv_ffn = w.vec(p + "canon2", {width, hc.conv_taps});
            Y.ffn_gate = w.mat(p + "mlp.gate", Y.ff, width);
            Y.ffn_up = w.mat(p + "mlp.up", Y.ff, width);
            Y.ffn_down = w.mat(p + "mlp.down", width, Y.ff);
        }
    }
    // what snapshots hold, per layer run in execution order
    for (uint32_t i = 0; i < hc.n_layers; ++i) {
        const bool looped = hc.loop_times && i >= hc.loop_start && i < hc.loop_stop;
        if (looped && i != hc.loop_start) continue;
        const uint32_t stop = looped ? hc.loop_stop : i + 1, times = looped ? hc.loop_times : 1;
        for (uint32_t t = 0; t < times; ++t)
            for (uint32_t j = i; j < stop; ++j) {
                const cera_hip_attn_spec& a = layers[j].attn;
                self->state_.push_back({static_cast<size_t>(a.kv_heads) * a.dim, static_cast<size_t>(a.kv_heads) * a.vdim,
                                        static_cast<size_t>(hc.conv_taps - 1) * width});
            }
    }
    const cera_hip_attn_spec& a0 = layers[0].attn;
    c.n_layers = self->state_.size();
    c.hidden_size = width;
    c.intermediate_size = layers[0].ff;
    c.n_heads = a0.heads;
    c.n_kv_heads = a0.kv_heads;
    c.head_dim = a0.dim;
    c.vocab_size = hc.vocab;
    c.max_seq_len = hc.max_seq_len;
    c.rope_theta = static_cast<float>(a0.rot_base);
    c.rms_norm_eps = hc.eps;
    c.scalars.residual = hc.residual_mult;
    c.scalars.attn = a0.scale;

    self->open_context(opt.device);
    if (cera_hip_layered_create(self->ctx_, &hc, layers.data(), &self->model_) != CERA_HIP_OK)
        bail(std::string("hip model: ") + cera_hip_last_error(self->ctx_));
    return self;
}

}  // namespace cera
