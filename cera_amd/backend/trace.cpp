#include "trace.h"

#include <algorithm>
#include <cstdio>
#include <cstdlib>
#include <cstring>
#include <fstream>
#include <iostream>
#include <map>

#include "json.h"
#include "load_model.h"

namespace cera {
namespace {

struct Request {
    InferenceState state;
    StateSnapshot parked;   // while another request has the model
};

const Json& need(const Json& o, const char* key, Json::Type type) {
    const Json* v = o.find(key);
    if (!v || v->type != type) throw BackendError(std::string("trace: a step needs \"") + key + "\"");
    return *v;
}
std::vector<uint32_t> numbers(const Json& a, const char* what) {
    std::vector<uint32_t> v;
    for (const Json& e : a.arr) {
        if (!e.is_int || e.integer < 0 || e.integer > 0x7FFFFFFF) throw BackendError(std::string("trace: bad number in ") + what);
        v.push_back(static_cast<uint32_t>(e.integer));
    }
    return v;
}

}  // namespace

void replay_trace(Model& model, std::istream& in, const std::string& out_dir) {
    const size_t vocab = model.config().vocab_size;
    std::map<std::string, Request> live;
    std::string on_device, line;   // name of the request whose state the model holds
    while (std::getline(in, line)) {
        if (line.find_first_not_of(" \t\r") == std::string::npos) continue;
        Json step;
        std::string err;
        if (!Json::parse(line, &step, &err)) throw BackendError("trace: " + err);
        const Json& number = need(step, "step", Json::Number);
        if (!number.is_int) throw BackendError("trace: step must be an integer");
        std::vector<float> wanted;
        for (const Json& entry : need(step, "entries", Json::Array).arr) {
            const std::string id = need(entry, "id", Json::String).str;
            const std::vector<uint32_t> tokens = numbers(need(entry, "tokens", Json::Array), "tokens");
            const std::vector<uint32_t> want = numbers(need(entry, "want", Json::Array), "want");
            if (tokens.empty()) throw BackendError("trace: an entry without tokens");
            for (uint32_t w : want)
                if (w >= tokens.size()) throw BackendError("trace: a wanted place beyond the entry's tokens");
            const bool fresh = live.count(id) == 0;
            Request& r = live[id];
            if (on_device != id) {
                auto held = live.find(on_device);
                if (!on_device.empty() && held != live.end()) held->second.parked = model.snapshot_state();
                if (!fresh) {
                    model.restore_state(r.parked);
                    r.parked = StateSnapshot();
                }
                on_device = id;   // a fresh one starts at position 0, which starts the model over
            }
            std::vector<float> logits;
            const size_t pos = r.state.seq_len;
            if (tokens.size() == 1) {
                logits = model.forward(tokens.data(), 1, pos, r.state);
            } else if (want.empty() || (want.size() == 1 && want[0] + 1 == tokens.size())) {
                logits = model.forward_prefill(tokens.data(), tokens.size(), pos, r.state);
                wanted.insert(wanted.end(), logits.begin(), logits.begin() + (want.empty() ? 0 : vocab));
                continue;
            } else {
                if (!model.supports_all_logits()) throw BackendError("trace: the model has no logits of every position");
                logits = model.forward_prefill_logits_all(tokens.data(), tokens.size(), pos, r.state);
            }
            for (uint32_t w : want) wanted.insert(wanted.end(), logits.begin() + w * vocab, logits.begin() + (w + 1) * vocab);
        }
        if (!wanted.empty()) {
            const std::string path = out_dir + "/" + std::to_string(number.integer) + ".f32";
            std::ofstream f(path, std::ios::binary);
            f.write(reinterpret_cast<const char*>(wanted.data()), static_cast<std::streamsize>(wanted.size() * sizeof(float)));
            f.close();
            if (!f) throw BackendError("trace: cannot write " + path);
        }
        for (const Json& e : need(step, "end", Json::Array).arr) {
            if (e.type != Json::String || !live.erase(e.str)) throw BackendError("trace: end of an unknown request");
            if (on_device == e.str) on_device.clear();
        }
        std::printf("done %lld\n", static_cast<long long>(number.integer));
        std::fflush(stdout);
    }
}

int trace_main(int argc, char** argv, int first) {
    std::map<std::string, std::string> a;
    for (int i = first; i < argc; i += 2) {
        if (std::strncmp(argv[i], "--", 2) != 0 || i + 1 >= argc) {
            std::fprintf(stderr, "unexpected argument: %s\n", argv[i]);
            return 2;
        }
        a[argv[i] + 2] = argv[i + 1];
    }
    for (const auto& kv : a)
        if (kv.first != "model" && kv.first != "out" && kv.first != "dtype" && kv.first != "max-tokens" && kv.first != "device") {
            std::fprintf(stderr, "unknown option: --%s\n", kv.first.c_str());
            return 2;
        }
    if (!a.count("model") || !a.count("out")) {
        std::fprintf(stderr, "usage: --model DIR --out DIR [--dtype bfloat16|float32] [--max-tokens N] [--device D]\n");
        return 2;
    }
    const std::string dtype = a.count("dtype") ? a["dtype"] : "bfloat16";
    if (dtype != "bfloat16" && dtype != "float32") {
        std::fprintf(stderr, "--dtype must be bfloat16 or float32\n");
        return 2;
    }
    try {
        LoadOptions opt;
        opt.f32 = dtype == "float32";
        opt.device = a.count("device") ? std::atoi(a["device"].c_str()) : 0;
        // one sequence can at most take all the live tokens; the model caps this at its own positions
        opt.context_size = a.count("max-tokens") ? std::max<size_t>(1, std::strtoull(a["max-tokens"].c_str(), nullptr, 10)) : SIZE_MAX;
        std::unique_ptr<Model> model = load_model_dir(a["model"], opt);
        replay_trace(*model, std::cin, a["out"]);
    } catch (const std::exception& e) {
        std::fprintf(stderr, "trace failed: %s\n", e.what());
        return 1;
    }
    return 0;
}

}  // namespace cera
