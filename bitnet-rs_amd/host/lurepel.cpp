// lurepel.cpp -- the Lurepel design: config.json and tensor names -> a StackModel.
//
// Grouped-head attention within chunks of positions whose values are the keys as projected: banded rotary positions on part of a head, queries and
// keys of unit root mean square, a sink of score zero, one gate per head.  The feed-forward is dense and gated, or a mixture of gated
// experts some of which hand their input through.  Norms stand behind the embedding and behind the sublayers, which read the residual stream itself.
// Fixed by the design: the tanh form of gelu in dense layers, silu in experts, choice by corrected scores, weights as the scores are.
#include <memory>

#include "registry.hpp"
#include "safetensors.hpp"
#include "stack_model.hpp"

namespace bitnet_host {

namespace {

void read_rotary(const JsonView &r, RotarySpec &rot) {
    rot.dims = r.integer("dims", 0), rot.base = r.number("base");
    if (!r.has("scaling")) return;
    const JsonView s = r.at("scaling");
    rot.banded = true;
    rot.factor = s.number("factor"), rot.original = s.number("original"), rot.slow = s.number("low"), rot.fast = s.number("high");
}

bool read_spec(const Json &config, StackSpec &s, std::string &err) {
    const JsonView c{&config, "", &err};
    s.width = c.integer("width");
    s.vocab = c.integer("vocab");
    s.eps = (float)c.at("norm").number("eps");
    const Json *layers = config.find("layers");
    if (!layers || layers->kind != Json::Array || layers->items.empty()) {
        if (err.empty()) err = "config: layers: missing array";
        return false;
    }
    for (size_t i = 0; i < layers->items.size() && err.empty(); ++i) {
        const JsonView l{&layers->items[i], "layers[" + std::to_string(i) + "].", &err};
        LayerSpec L;
        L.mixer = LayerSpec::Attention;
        const std::string type = l.text("type");
        if (type != "attention" && err.empty()) err = "config: " + l.path + "type: unknown mixer '" + type + "'";
        const JsonView m = l.at("mixer");
        AttentionSpec &a = L.attention;
        a.heads = m.integer("heads"), a.kv_heads = m.integer("kv_heads"), a.dim = m.integer("dim"), a.vdim = m.integer("vdim");
        a.scale = (float)m.number("scale");
        a.unit_norm = a.values_are_keys = a.head_gate = true;
        if (m.has("rot")) read_rotary(m.at("rot"), a.rot);
        if (m.has("mask")) a.chunk = m.at("mask").integer("size");
        if (l.has("mlp")) {
            const JsonView f = l.at("mlp");
            const std::string kind = f.text("kind");
            if (kind == "dense") {
                L.ff = f.integer("ff");
                L.act_ff = BITNET_HIP_ACT_GELU_TANH, L.gated = true;
            } else if (kind == "moe") {
                const JsonView r = f.at("router");
                ExpertsSpec &e = L.experts;
                e.count = r.integer("experts"), e.top = r.integer("top"), e.ff = f.at("expert").integer("ff");
                if (r.has("identity")) e.identity = r.integer("identity", 0);
                e.act = BITNET_HIP_ACT_SILU, e.gated = e.raw = true;
            } else if (err.empty()) {
                err = "config: " + f.path + "kind: unknown feed-forward '" + kind + "'";
            }
        }
        s.layers.push_back(L);
    }
    return err.empty();
}

bool read_layer(const SafeTensors &t, const StackSpec &s, size_t i, StackLayerWeights &w, std::string &err) {
    const std::string p = "l" + std::to_string(i) + ".", m = p + "mix.", f = p + "mlp.";
    const size_t W = s.width;
    const LayerSpec &L = s.layers[i];
    const AttentionSpec &a = L.attention;
    const ExpertsSpec &e = L.experts;
    auto mat = [&](const std::string &name, const uint16_t **dst, size_t rows, size_t cols) { return (*dst = t.matrix(name, rows, cols, err)) != nullptr; };
    bool ok = t.vector(p + "norm1", W, w.norm1b, err) && mat(m + "q", &w.q, (size_t)a.heads * a.dim, W) && mat(m + "k", &w.k, (size_t)a.kv_heads * a.dim, W) &&
              mat(m + "g", &w.g, a.heads, W) && mat(m + "o", &w.o, W, (size_t)a.heads * a.vdim);
    w.sink.assign(a.heads, 0.f);
    if (ok && (L.ff > 0 || e.count > 0)) ok = t.vector(p + "norm2", W, w.norm2b, err);
    if (ok && L.ff > 0) ok = mat(f + "gate", &w.gate, L.ff, W) && mat(f + "up", &w.up, L.ff, W) && mat(f + "down", &w.down, W, L.ff);
    if (ok && e.count > 0) {
        const size_t outputs = (size_t)e.count + e.identity;
        ok = mat(f + "router", &w.router, outputs, W) && t.vector(f + "correction", outputs, w.router_correction, err);
        w.expert_gate.resize(e.count), w.expert_up.resize(e.count), w.expert_down.resize(e.count);
        for (int k = 0; ok && k < e.count; ++k) {
            const std::string x = f + "e" + std::to_string(k) + ".";
            ok = mat(x + "gate", &w.expert_gate[k], e.ff, W) && mat(x + "up", &w.expert_up[k], e.ff, W) && mat(x + "down", &w.expert_down[k], W, e.ff);
        }
    }
    return ok;
}

Sequence *open_lurepel(const Json &config, const std::string &dir, const OpenOptions &opt, std::string &err) {
    StackSpec s;
    SafeTensors t;
    if (!read_spec(config, s, err) || !t.open(dir + "/model.safetensors", err)) return nullptr;
    std::unique_ptr<StackModel> model(new StackModel(s, opt.f32, opt.max_pos));
    auto failed = [&] {
        if (err.empty()) err = model->error();
        return nullptr;
    };
    if (model->dead()) return failed();
    for (size_t i = 0; i < s.layers.size(); ++i) {
        StackLayerWeights w;
        if (!read_layer(t, s, i, w, err) || model->set_layer((int)i, w) != 0) return failed();
    }
    StackGlobalWeights g;
    g.embed = t.matrix("embed", s.vocab, s.width, err), g.head = g.embed ? t.matrix("head", s.vocab, s.width, err) : nullptr;
    if (!g.head || !t.vector("embed.norm", s.width, g.embed_norm, err) || !t.vector("final.norm", s.width, g.final_norm, err) || model->set_globals(g) != 0)
        return failed();
    return model.release();
}

const RegisterArchitecture kLurepel("Lurepel", open_lurepel);

}  // namespace

}  // namespace bitnet_host
