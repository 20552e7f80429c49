// The Nafevik architecture: config.json and tensor names -> cera_hip_layered_create.
//
// Embedding plus learned positions; parallel attention and gated feed-forward behind one RMS norm, each reading its
// input through a short causal convolution; sigmoid attention inside chunks, with YaRN rotation in adjacent pairs and
// a gate per head; a range of layers run several times, each pass starting from a product over the residual and the
// embedding.
#include <algorithm>

#include "layered_reader.h"

namespace cera {
namespace layered {
namespace {

cera_hip_attn_spec read_attention(const ConfigNode& m) {
    cera_hip_attn_spec a{};
    a.heads = m.at("heads").u32();
    a.kv_heads = m.at("kv_heads").u32();
    a.dim = m.at("dim").u32();
    a.vdim = m.at("vdim").u32();
    a.scale = static_cast<float>(m.at("scale").num());
    if (m.has("mask")) a.chunk = m.at("mask").at("size").u32();
    if (m.has("rot")) {
        const ConfigNode r = m.at("rot");
        a.rot_dims = r.at("dims").u32(0);
        a.rot_base = r.at("base").num();
        if (r.has("scaling")) {
            const ConfigNode s = r.at("scaling");
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

void read_nafevik(const ConfigNode& top, size_t context, Description& d, ModelConfig& c) {
    LayeredWeights& w = d.weights;
    cera_hip_layered_config& hc = d.config;
    hc.block = CERA_HIP_BLOCK_PARALLEL;
    hc.width = top.at("width").u32();
    hc.vocab = top.at("vocab").u32();
    hc.conv_taps = top.at("canon").at("taps").u32();
    hc.eps = static_cast<float>(top.at("norm").at("eps").num());
    hc.residual_mult = static_cast<float>(top.at("residual_mult").num());
    const uint32_t positions = top.at("max_positions").u32();
    hc.max_seq_len = static_cast<uint32_t>(std::min<size_t>(context, positions));
    const std::vector<ConfigNode> list = read_layers(top, d);
    const uint64_t width = hc.width;
    hc.embed = w.mat("embed", hc.vocab, width);
    hc.pos = w.mat("pos", positions, width);
    hc.head = w.mat("head", hc.vocab, width);
    hc.final_norm = w.vec("final.norm", {width});
    if (top.has("loop")) {
        const ConfigNode l = top.at("loop");
        hc.loop_start = l.at("start").u32(0);
        hc.loop_stop = l.at("stop").u32();
        hc.loop_times = l.at("times").u32();
        if (hc.loop_start >= hc.loop_stop || hc.loop_stop > hc.n_layers) bail("config.json: loop.start / loop.stop are no range of layers");
        hc.loop_in = w.mat("loop.in", width, 2 * width);
        hc.loop_step = w.vec("loop.step", {hc.loop_times, width});
    }

    for (uint32_t i = 0; i < hc.n_layers; ++i) {
        const ConfigNode& l = list[i];
        const std::string p = "l" + std::to_string(i) + ".";
        cera_hip_layered_layer& Y = d.layers[i];
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
            const ConfigNode f = l.at("mlp");
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
                const cera_hip_attn_spec& a = d.layers[j].attn;
                d.state.push_back({static_cast<size_t>(a.kv_heads) * a.dim, static_cast<size_t>(a.kv_heads) * a.vdim,
                                        static_cast<size_t>(hc.conv_taps - 1) * width});
            }
    }
    const cera_hip_attn_spec& a0 = d.layers[0].attn;
    c.n_layers = d.state.size();
    c.hidden_size = width;
    c.intermediate_size = d.layers[0].ff;
    c.n_heads = a0.heads;
    c.n_kv_heads = a0.kv_heads;
    c.head_dim = a0.dim;
    c.vocab_size = hc.vocab;
    c.max_seq_len = hc.max_seq_len;
    c.rope_theta = static_cast<float>(a0.rot_base);
    c.rms_norm_eps = hc.eps;
    c.scalars.residual = hc.residual_mult;
    c.scalars.attn = a0.scale;
}

}  // namespace layered
}  // namespace cera
