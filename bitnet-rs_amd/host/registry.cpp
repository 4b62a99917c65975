// registry.cpp -- see registry.hpp.
#include "registry.hpp"

#include <fstream>
#include <map>
#include <sstream>

namespace bitnet_host {

namespace {
std::map<std::string, ArchitectureFactory> &architectures() {
    static std::map<std::string, ArchitectureFactory> m;
    return m;
}
std::map<std::string, FileFactory> &formats() {
    static std::map<std::string, FileFactory> m;
    return m;
}
}  // namespace

RegisterArchitecture::RegisterArchitecture(const char *name, ArchitectureFactory make) { architectures()[name] = make; }
RegisterFileFormat::RegisterFileFormat(const char *suffix, FileFactory make) { formats()[suffix] = make; }

std::vector<std::string> registered_names() {
    std::vector<std::string> v;
    for (const auto &a : architectures()) v.push_back(a.first);
    for (const auto &f : formats()) v.push_back(f.first);
    return v;
}

Sequence *open_model(const std::string &path, const OpenOptions &opt, std::string &err) {
    if (opt.max_pos < 2 || opt.max_pos > (1 << 22)) {
        err = "max_pos out of range";
        return nullptr;
    }
    for (const auto &f : formats())
        if (path.size() > f.first.size() && path.compare(path.size() - f.first.size(), f.first.size(), f.first) == 0) return f.second(path, opt, err);
    std::ifstream in(path + "/config.json", std::ios::binary);
    if (!in) {
        err = path + ": neither a known file format nor a folder with config.json";
        return nullptr;
    }
    std::stringstream ss;
    ss << in.rdbuf();
    const std::string text = ss.str();
    Json config;
    if (!Json::parse(text.data(), text.size(), config, err)) return nullptr;
    const Json *arch = config.find("architecture");
    const auto it = arch ? architectures().find(arch->str) : architectures().end();
    if (it == architectures().end()) {
        err = "config.json: architecture '" + (arch ? arch->str : std::string()) + "' is not registered";
        return nullptr;
    }
    return it->second(config, path, opt, err);
}

}  // namespace bitnet_host

using bitnet_host::Sequence;

static thread_local std::string g_open_error;

#define SEQ(rc)                                 \
    Sequence *S = static_cast<Sequence *>(d);   \
    if (!S || S->dead()) return rc

extern "C" {
void *bitnet_host_open_model(const char *path, int f32, int max_pos) {
    g_open_error.clear();
    try {
        bitnet_host::OpenOptions o;
        o.f32 = f32 != 0;
        o.max_pos = max_pos;
        return path ? bitnet_host::open_model(path, o, g_open_error) : nullptr;
    } catch (const std::exception &e) {
        g_open_error = e.what();
        return nullptr;
    }
}
const char *bitnet_host_open_error(void) { return g_open_error.c_str(); }
const char *bitnet_host_registered(void) {
    static thread_local std::string s;
    s.clear();
    for (const auto &n : bitnet_host::registered_names()) s += (s.empty() ? "" : ",") + n;
    return s.c_str();
}
void bitnet_host_destroy(void *d) { delete static_cast<Sequence *>(d); }
const char *bitnet_host_error(void *d) { return d ? static_cast<Sequence *>(d)->error().c_str() : "null decoder"; }
int bitnet_host_vocab(void *d) { SEQ(-1); return S->vocab(); }
int bitnet_host_width(void *d) { SEQ(-1); return S->width(); }
int bitnet_host_reset(void *d) { SEQ(BITNET_HIP_ERR_INVALID_ARGUMENT); return S->reset(); }
int bitnet_host_feed(void *d, const int32_t *tokens, int n) { SEQ(BITNET_HIP_ERR_INVALID_ARGUMENT); return S->feed(tokens, n); }
int bitnet_host_run(void *d, int n, int with_logits, int use_graph, float *elapsed_ms) {
    SEQ(BITNET_HIP_ERR_INVALID_ARGUMENT);
    return S->run(n, with_logits != 0, use_graph != 0, elapsed_ms);
}
int bitnet_host_prefill(void *d, int n, int with_logits, int digits, float *elapsed_ms) {
    SEQ(BITNET_HIP_ERR_INVALID_ARGUMENT);
    return S->prefill(n, with_logits != 0, digits, elapsed_ms);
}
int bitnet_host_forward(void *d, const int32_t *tokens, int n, const int32_t *want, int n_want, float *logits) {
    SEQ(BITNET_HIP_ERR_INVALID_ARGUMENT);
    return S->forward(tokens, n, want, n_want, logits);
}
int bitnet_host_prepare_graphs(void *d, int with_logits) { SEQ(BITNET_HIP_ERR_INVALID_ARGUMENT); return S->prepare_graphs(with_logits != 0); }
int bitnet_host_position(void *d) { SEQ(-1); return S->position(); }
int bitnet_host_history(void *d, int32_t *out, int n) { SEQ(BITNET_HIP_ERR_INVALID_ARGUMENT); return S->history(out, n); }
int bitnet_host_last_logits(void *d, float *out) { SEQ(BITNET_HIP_ERR_INVALID_ARGUMENT); return S->last_logits(out); }
int bitnet_host_last_hidden(void *d, float *out) { SEQ(BITNET_HIP_ERR_INVALID_ARGUMENT); return S->last_hidden(out); }
uint64_t bitnet_host_weight_bytes(void *d) { SEQ(0); return S->weight_bytes(); }
}
