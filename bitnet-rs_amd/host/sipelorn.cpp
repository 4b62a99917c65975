// sipelorn.cpp -- the Sipelorn design: config.json and tensor names -> a StackModel.
//
// Layers of two kinds behind layer norms: grouped-head attention within a window (queries, keys and values with biases and short convolutions over
// time, no rotation but a penalty on the score that grows with the logarithm of the distance, a gate per output column, keys and values of an earlier layer
// in some) and latent attention (queries straight from the input, neighbouring elements of a part of its own turn, YaRN).  The feed-forward is dense
// with xIELU, a mixture of gated experts chosen within groups beside a shared expert with a number of its own per token, or absent.  What a sublayer adds is
// gated column by column, and behind the sublayers every layer adds an input of the token's own.  The embedding adds a row for the pair of the previous and
// the current token.  Fixed by the design: silu in experts, sigmoid scores, weights as the scores are, the tanh form of gelu on the token's input.
#include <algorithm>
#include <cmath>
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
    rot.yarn = true;
    rot.factor = s.number("factor"), rot.original = s.number("original"), rot.fast = s.number("fast"), rot.slow = s.number("slow");
}

void read_mixer(const JsonView &l, LayerSpec &L) {
    const std::string type = l.text("type");
    const JsonView m = l.at("mixer");
    if (type == "attention") {
        L.mixer = LayerSpec::Attention;
        AttentionSpec &a = L.attention;
        a.heads = m.integer("heads"), a.kv_heads = m.integer("kv_heads"), a.dim = m.integer("dim"), a.vdim = m.integer("vdim");
        a.scale = (float)m.number("scale");
        a.taps = m.integer("conv");
        if (m.has("mask")) a.window = m.at("mask").integer("size");
        if (m.has("kv_from")) a.kv_from = m.integer("kv_from", 0);
        a.far_penalty = a.column_gate = true;
    } else if (type == "latent_attention") {
        L.mixer = LayerSpec::Latent;
        LatentSpec &a = L.latent;
        a.heads = m.integer("heads"), a.dim = m.integer("dim"), a.rot_dim = m.integer("rot_dim"), a.vdim = m.integer("vdim"), a.kv_rank = m.integer("kv_rank");
        a.scale = (float)m.number("scale");
        a.neighbours = true;
        read_rotary(m.at("rot"), a.rot);
    } else if (l.err->empty()) {
        *l.err = "config: " + l.path + "type: unknown mixer '" + type + "'";
    }
}

void read_mlp(const JsonView &f, LayerSpec &L) {
    const std::string kind = f.text("kind");
    if (kind == "dense") {
        L.ff = f.integer("ff");
        L.act_ff = BITNET_HIP_ACT_XIELU;
    } else if (kind == "moe") {
        const JsonView r = f.at("router");
        ExpertsSpec &e = L.experts;
        e.count = r.integer("experts"), e.top = r.integer("top"), e.ff = f.at("expert").integer("ff");
        e.act = BITNET_HIP_ACT_SILU, e.gated = e.raw = e.sigmoid = true;
        if (r.has("groups")) {
            const JsonView g = r.at("groups");
            e.groups = g.integer("count"), e.keep = g.integer("keep");
        }
        if (f.has("shared")) {
            L.ff = f.at("shared").integer("ff");
            L.act_ff = BITNET_HIP_ACT_SILU, L.gated = L.shared_gate = true;
        }
    } else if (f.err->empty()) {
        *f.err = "config: " + f.path + "kind: unknown feed-forward '" + kind + "'";
    }
}

bool read_spec(const Json &config, StackSpec &s, std::string &err) {
    const JsonView c{&config, "", &err};
    s.width = c.integer("width");
    s.vocab = c.integer("vocab");
    s.eps = (float)c.at("norm").number("eps");
    s.center = s.residual_gate = true;
    const JsonView embedding = c.at("embedding");
    s.embed_scale = (float)embedding.number("scale");
    if (embedding.has("bigram")) {
        const JsonView b = embedding.at("bigram");
        s.pairs.buckets = (uint64_t)b.integer("buckets"), s.pairs.mul_prev = (uint64_t)b.integer("mul_prev", 0, 0x7fffffff);
        s.pairs.mul_cur = (uint64_t)b.integer("mul_cur", 0, 0x7fffffff);
    }
    if (c.has("token_side")) s.side_dim = c.at("token_side").integer("dim");
    const Json *layers = config.find("layers");
    if (!layers || layers->kind != Json::Array || layers->items.empty()) {
        if (err.empty()) err = "config: layers: missing array";
        return false;
    }
    for (size_t i = 0; i < layers->items.size() && err.empty(); ++i) {
        const JsonView l{&layers->items[i], "layers[" + std::to_string(i) + "].", &err};
        LayerSpec L;
        read_mixer(l, L);
        if (l.has("mlp")) read_mlp(l.at("mlp"), L);
        s.layers.push_back(L);
    }
    return err.empty();
}

bool read_layer(const SafeTensors &t, const StackSpec &s, size_t i, StackLayerWeights &w, std::string &err) {
    const std::string p = "l" + std::to_string(i) + ".", m = p + "mix.", f = p + "mlp.";
    const size_t W = s.width;
    const LayerSpec &L = s.layers[i];
    const ExpertsSpec &e = L.experts;
    auto mat = [&](const std::string &name, const uint16_t **dst, size_t rows, size_t cols) { return (*dst = t.matrix(name, rows, cols, err)) != nullptr; };
    auto vec = [&](const std::string &name, std::vector<float> &dst, size_t n) { return t.vector(name, n, dst, err); };
    auto convolved = [&](const std::string &name, const uint16_t **dst, std::vector<float> &bias, std::vector<float> &taps, size_t rows) {
        const uint16_t *src = mat(name, dst, rows, W) && vec(name + ".b", bias, rows) ? t.matrix(name + ".conv", rows, L.attention.taps, err) : nullptr;
        for (size_t k = 0; src && k < rows * L.attention.taps; ++k) taps.push_back(bf16_value(src[k]));
        return src != nullptr;
    };
    bool ok = vec(p + "norm1", w.norm1, W) && vec(p + "norm1.b", w.norm1_bias, W) && mat(p + "rg1", &w.rg1, W, W) && vec(p + "rg1.b", w.rg1_b, W);
    if (L.mixer == LayerSpec::Attention) {
        const AttentionSpec &a = L.attention;
        const size_t H = a.heads, G = a.kv_heads, D = a.dim, V = a.vdim;
        ok = ok && convolved(m + "q", &w.q, w.q_b, w.q_conv, H * D);
        if (a.kv_from < 0) ok = ok && convolved(m + "k", &w.k, w.k_b, w.k_conv, G * D) && convolved(m + "v", &w.v, w.v_b, w.v_conv, G * V);
        ok = ok && vec(m + "r1", w.far_weight, H) && vec(m + "r2", w.far_rate, H) && mat(m + "g", &w.g, H * V, W) && mat(m + "o", &w.o, W, H * V);
    } else {
        const LatentSpec &a = L.latent;
        const size_t H = a.heads, D = a.dim, R = a.rot_dim, V = a.vdim, C = a.kv_rank;
        ok = ok && mat(m + "q", &w.q, H * (D + R), W) && mat(m + "dkv", &w.dkv, C + R, W) && vec(m + "dkv.norm", w.dkv_norm, C) && mat(m + "uk", &w.uk, H * D, C) &&
             mat(m + "uv", &w.uv, H * V, C) && mat(m + "o", &w.o, W, H * V);
    }
    if (L.ff > 0 || e.count > 0)
        ok = ok && vec(p + "norm2", w.norm2, W) && vec(p + "norm2.b", w.norm2_bias, W) && mat(p + "rg2", &w.rg2, W, W) && vec(p + "rg2.b", w.rg2_b, W);
    if (L.ff > 0 && e.count == 0) {
        std::vector<float> act;
        ok = ok && mat(f + "up", &w.up, L.ff, W) && mat(f + "down", &w.down, W, L.ff) && vec(f + "act", act, 2);
        auto softplus = [](double z) { return std::max(z, 0.0) + std::log1p(std::exp(-std::fabs(z))); };
        if (ok) w.act_a = (float)softplus(act[0]), w.act_b = (float)(0.5 + softplus(act[1]));
    }
    if (e.count > 0) {
        ok = ok && mat(f + "router", &w.router, e.count, W) && vec(f + "correction", w.router_correction, e.count);
        if (L.ff > 0)
            ok = ok && mat(f + "shared.gate", &w.gate, L.ff, W) && mat(f + "shared.up", &w.up, L.ff, W) && mat(f + "shared.down", &w.down, W, L.ff) &&
                 mat(f + "shared.sg", &w.shared_gate, 1, W);
        w.expert_gate.resize(e.count), w.expert_up.resize(e.count), w.expert_down.resize(e.count);
        for (int k = 0; ok && k < e.count; ++k) {
            const std::string x = f + "e" + std::to_string(k) + ".";
            ok = mat(x + "gate", &w.expert_gate[k], e.ff, W) && mat(x + "up", &w.expert_up[k], e.ff, W) && mat(x + "down", &w.expert_down[k], W, e.ff);
        }
    }
    if (s.side_dim > 0)
        ok = ok && mat(p + "side.gate", &w.side_gate, s.side_dim, W) && mat(p + "side.proj", &w.side_proj, W, s.side_dim) && vec(p + "side.norm", w.side_norm, W);
    return ok;
}

Sequence *open_sipelorn(const Json &config, const std::string &dir, const OpenOptions &opt, std::string &err) {
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
    auto mat = [&](const std::string &name, const uint16_t **dst, size_t rows, size_t cols) { return (*dst = t.matrix(name, rows, cols, err)) != nullptr; };
    if (!mat("embed", &g.embed, s.vocab, s.width) || !mat("head", &g.head, s.vocab, s.width) || !t.vector("final.norm", s.width, g.final_norm, err) ||
        !t.vector("final.norm.b", s.width, g.final_bias, err) || (s.pairs.buckets > 0 && !mat("bigram", &g.pairs, s.pairs.buckets + 1, s.width)) ||
        (s.side_dim > 0 && !mat("side.embed", &g.side, s.vocab, s.layers.size() * (size_t)s.side_dim)) || model->set_globals(g) != 0)
        return failed();
    return model.release();
}

const RegisterArchitecture kSipelorn("Sipelorn", open_sipelorn);

}  // namespace

}  // namespace bitnet_host
