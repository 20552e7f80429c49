// The Fidinex architecture: config.json and tensor names -> cera_hip_layered_create.
//
// Mixer and feed-forward one after the other behind an RMS norm each, over several residual streams that every
// sublayer reads and writes with its own weights; per layer either attention over cached latents (one latent and one
// rotated key part per token) or attention with grouped heads, without rotation but with norms on queries and keys,
// queries that grow with the position and values mixed with those of the first such layer; a sink per head in every
// softmax; squared-relu feed-forwards; the embedding is the output matrix.
#include <algorithm>

#include "layered_reader.h"

namespace cera {
namespace layered {
namespace {

// positions of a model whose config.json and caller name none
constexpr size_t DEFAULT_POSITIONS = 32768;

cera_hip_attn_spec read_softmax(const ConfigNode& m) {
    cera_hip_attn_spec a{};
    a.kind = CERA_HIP_MIXER_SOFTMAX;
    a.kv_heads = m.at("kv_heads").u32();
    if (m.has("q_temp")) {
        a.q_temp_coef = m.at("q_temp").at("coef").num();
        a.q_temp_every = m.at("q_temp").at("every").num();
        if (a.q_temp_every <= 0) bail("config.json: " + m.path + "q_temp.every must be positive");
    }
    a.v_mix = m.has("v_mix") && m.at("v_mix").flag() ? 1 : 0;
    return a;
}
cera_hip_attn_spec read_latent(const ConfigNode& m) {
    cera_hip_attn_spec a{};
    a.kind = CERA_HIP_MIXER_LATENT;
    a.rot_dim = m.at("rot_dim").u32();
    a.kv_rank = m.at("kv_rank").u32();
    a.rot_dims = m.at("rot").at("dims").u32(0);
    a.rot_base = m.at("rot").at("base").num();
    return a;
}

}  // namespace

void read_fidinex(const ConfigNode& top, size_t context, Description& d, ModelConfig& c) {
    LayeredWeights& w = d.weights;
    cera_hip_layered_config& hc = d.config;
    hc.block = CERA_HIP_BLOCK_SEQUENTIAL;
    hc.width = top.at("width").u32();
    hc.vocab = top.at("vocab").u32();
    hc.streams = top.has("streams") ? top.at("streams").u32() : 1;
    hc.eps = static_cast<float>(top.at("norm").at("eps").num());
    hc.max_seq_len = static_cast<uint32_t>(context == SIZE_MAX ? DEFAULT_POSITIONS : std::min<size_t>(context, 0x7FFFFFFF));
    const uint64_t width = hc.width, S = hc.streams;
    hc.embed = hc.head = w.mat("embed", hc.vocab, width);
    hc.final_norm = w.vec("final.norm", {width});
    // how a sublayer reads and writes the streams; a model without the key has one, read and written as it is
    auto streams = [&](const std::string& p) {
        if (!top.has("streams")) return w.keep({1.0f, 1.0f, 1.0f});
        return w.join({w.vec(p + "in", {S}), w.vec(p + "out", {S}), w.vec(p + "mix", {S, S})}, {S, S, S * S});
    };
    const std::vector<ConfigNode> list = read_layers(top, d);
    for (uint32_t i = 0; i < hc.n_layers; ++i) {
        const ConfigNode& l = list[i];
        const std::string p = "l" + std::to_string(i) + ".";
        cera_hip_layered_layer& Y = d.layers[i];
        const ConfigNode m = l.at("mixer");
        const std::string& type = l.at("type").str();
        if (type == "latent_attention") Y.attn = read_latent(m);
        else if (type == "attention") Y.attn = read_softmax(m);
        else bail("config.json: " + l.path + "type: no mixer " + type);
        cera_hip_attn_spec& a = Y.attn;
        a.heads = m.at("heads").u32();
        a.dim = m.at("dim").u32();
        a.vdim = m.at("vdim").u32();
        a.scale = static_cast<float>(m.at("scale").num());
        const uint64_t H = a.heads, G = a.kv_heads, rank = a.kv_rank;
        Y.norm = w.vec(p + "norm1", {width});
        Y.streams_attn = streams(p + "hc1.");
        Y.sink = w.vec(p + "mix.sink", {H});
        Y.o = w.mat(p + "mix.o", width, H * a.vdim);
        if (a.kind == CERA_HIP_MIXER_LATENT) {
            Y.q = w.mat(p + "mix.q", H * (a.dim + a.rot_dim), width);
            Y.kv_down = w.mat(p + "mix.dkv", rank + a.rot_dim, width);
            Y.latent_norm = w.vec(p + "mix.dkv.norm", {rank});
            Y.k_up = w.mat(p + "mix.uk", H * a.dim, rank);
            Y.v_up = w.mat(p + "mix.uv", H * a.vdim, rank);
            d.state.push_back({static_cast<size_t>(rank), static_cast<size_t>(a.rot_dim), 0});
        } else {
            Y.q = w.mat(p + "mix.q", H * a.dim, width);
            Y.k = w.mat(p + "mix.k", G * a.dim, width);
            Y.v = w.mat(p + "mix.v", G * a.vdim, width);
            Y.q_norm = w.vec(p + "mix.q.norm", {a.dim});
            Y.k_norm = w.vec(p + "mix.k.norm", {a.dim});
            if (a.v_mix) Y.v_mix_lambda = *w.vec(p + "mix.vmix", {});
            d.state.push_back({static_cast<size_t>(G) * a.dim, static_cast<size_t>(G) * a.vdim, 0});
        }
        if (l.has("mlp")) {
            const ConfigNode f = l.at("mlp");
            if (f.at("kind").str() != "dense") bail("config.json: " + f.path + "kind: no feed-forward " + f.at("kind").str());
            Y.ff = f.at("ff").u32();
            Y.norm_ffn = w.vec(p + "norm2", {width});
            Y.streams_ffn = streams(p + "hc2.");
            Y.ffn_up = w.mat(p + "mlp.up", Y.ff, width);
            Y.ffn_down = w.mat(p + "mlp.down", width, Y.ff);
        }
    }
    const cera_hip_attn_spec& a0 = d.layers[0].attn;
    c.n_layers = d.state.size();
    c.hidden_size = width;
    c.intermediate_size = d.layers[0].ff;
    c.n_heads = a0.heads;
    c.n_kv_heads = a0.kind == CERA_HIP_MIXER_LATENT ? a0.heads : a0.kv_heads;
    c.head_dim = a0.dim + a0.rot_dim;
    c.vocab_size = hc.vocab;
    c.max_seq_len = hc.max_seq_len;
    c.rope_theta = static_cast<float>(a0.rot_base);
    c.rms_norm_eps = hc.eps;
    c.scalars.attn = a0.scale;
}

}  // namespace layered
}  // namespace cera
