// mimolix.cpp -- the Mimolix design: config.json and tensor names -> a StackModel.
//
// Layers of two kinds, each with its feed-forward side by side behind one layer norm: differential attention (two softmax maps per head over
// the same values, no positions but a temperature on the query) and the gated delta rule; the feed-forward is a mixture of experts with one
// expert shared by every token.  A range of layers runs several times, every pass entered through a projection of the stream and the embedding
// output.  Fixed by the design: silu behind the convolutions, square of relu in the experts, 1e-6 in the unit norms.
#include <memory>

#include "registry.hpp"
#include "safetensors.hpp"
#include "stack_model.hpp"

namespace bitnet_host {

namespace {

bool read_spec(const Json &config, StackSpec &s, std::string &err) {
    const JsonView c{&config, "", &err};
    s.width = c.integer("width");
    s.vocab = c.integer("vocab");
    s.eps = (float)c.at("norm").number("eps");
    s.center = true;
    s.embed_scale = (float)c.at("embedding").number("scale");
    s.residual_mult = (float)c.number("residual_mult");
    if (c.has("loop")) {
        const JsonView l = c.at("loop");
        s.loop.start = l.integer("start", 0), s.loop.stop = l.integer("stop"), s.loop.times = l.integer("times");
    }
    const Json *layers = config.find("layers");
    if (!layers || layers->kind != Json::Array || layers->items.empty()) {
        if (err.empty()) err = "config: layers: missing array";
        return false;
    }
    for (size_t i = 0; i < layers->items.size() && err.empty(); ++i) {
        const JsonView l{&layers->items[i], "layers[" + std::to_string(i) + "].", &err};
        LayerSpec L;
        L.parallel = true;
        const std::string type = l.text("type");
        const JsonView m = l.at("mixer");
        if (type == "attention") {
            L.mixer = LayerSpec::Attention;
            AttentionSpec &a = L.attention;
            a.heads = m.integer("heads"), a.kv_heads = m.integer("kv_heads"), a.dim = m.integer("dim"), a.vdim = m.integer("vdim");
            a.maps = 2;
            a.scale = (float)m.number("scale"), a.diff = (float)m.number("diff");
            if (m.has("q_temp")) {
                const JsonView t = m.at("q_temp");
                a.temp_coef = t.number("coef"), a.temp_every = t.number("every");
            }
        } else if (type == "delta") {
            L.mixer = LayerSpec::Delta;
            DeltaSpec &d = L.delta;
            d.heads = m.integer("heads"), d.kv_heads = m.integer("kv_heads"), d.dim = m.integer("dim"), d.vdim = m.integer("vdim"), d.taps = m.integer("conv");
        } else if (err.empty()) {
            err = "config: " + l.path + "type: unknown mixer '" + type + "'";
        }
        if (l.has("mlp")) {
            const JsonView f = l.at("mlp");
            if (err.empty() && f.text("kind") != "moe") err = "config: " + f.path + "kind: unknown feed-forward";
            const JsonView r = f.at("router");
            L.experts.count = r.integer("experts"), L.experts.top = r.integer("top"), L.experts.scale = (float)r.number("scale");
            L.experts.ff = f.at("expert").integer("ff");
            L.experts.act = L.act_ff = BITNET_HIP_ACT_RELU2;
            if (f.has("shared")) L.ff = f.at("shared").integer("ff");
        }
        s.layers.push_back(L);
    }
    return err.empty();
}

bool read_layer(const SafeTensors &t, const StackSpec &s, size_t i, StackLayerWeights &w, std::string &err) {
    const std::string p = "l" + std::to_string(i) + ".", m = p + "mix.", f = p + "mlp.";
    const size_t W = s.width;
    const LayerSpec &L = s.layers[i];
    auto mat = [&](const std::string &name, const uint16_t **dst, size_t rows, size_t cols) { return (*dst = t.matrix(name, rows, cols, err)) != nullptr; };
    auto vec = [&](const std::string &name, std::vector<float> &dst, size_t n) { return t.vector(name, n, dst, err); };
    auto taps = [&](const std::string &name, std::vector<float> &dst, size_t channels, size_t n) {
        const uint16_t *src = t.matrix(name, channels, n, err);
        for (size_t k = 0; src && k < channels * n; ++k) dst.push_back(bf16_value(src[k]));
        return src != nullptr;
    };
    bool ok = vec(p + "norm1", w.norm1, W) && vec(p + "norm1.b", w.norm1_bias, W);
    if (L.mixer == LayerSpec::Attention) {
        const AttentionSpec &a = L.attention;
        const size_t D = a.dim;
        ok = ok && mat(m + "q", &w.q, a.heads * 2 * D, W) && mat(m + "k", &w.k, a.kv_heads * 2 * D, W) && mat(m + "v", &w.v, (size_t)a.kv_heads * a.vdim, W) &&
             vec(m + "q.norm", w.q_norm, D) && vec(m + "k.norm", w.k_norm, D) && vec(m + "lq1", w.lq1, D) && vec(m + "lk1", w.lk1, D) && vec(m + "lq2", w.lq2, D) &&
             vec(m + "lk2", w.lk2, D) && mat(m + "o", &w.o, W, (size_t)a.heads * a.vdim);
    } else {
        const DeltaSpec &d = L.delta;
        const size_t H = d.heads, qk = (size_t)d.kv_heads * d.dim, v = H * d.vdim, T = d.taps;
        ok = ok && mat(m + "q", &w.q, qk, W) && mat(m + "k", &w.k, qk, W) && mat(m + "v", &w.v, v, W) && taps(m + "q.conv", w.q_conv, qk, T) &&
             taps(m + "k.conv", w.k_conv, qk, T) && taps(m + "v.conv", w.v_conv, v, T) && mat(m + "b", &w.b, H, W) && mat(m + "a", &w.a, H, W) &&
             vec(m + "A_log", w.a_log, H) && vec(m + "dt_bias", w.dt_bias, H) && vec(m + "norm", w.out_norm, d.vdim) && mat(m + "g", &w.g, v, W) && mat(m + "o", &w.o, W, v);
    }
    const ExpertsSpec &e = L.experts;
    if (e.count > 0) {
        ok = ok && mat(f + "router", &w.router, e.count, W);
        if (L.ff > 0) ok = ok && mat(f + "shared.up", &w.up, L.ff, W) && mat(f + "shared.down", &w.down, W, L.ff);
        w.expert_up.resize(e.count), w.expert_down.resize(e.count);
        for (int k = 0; ok && k < e.count; ++k) {
            const std::string x = f + "e" + std::to_string(k) + ".";
            ok = mat(x + "up", &w.expert_up[k], e.ff, W) && mat(x + "down", &w.expert_down[k], W, e.ff);
        }
    }
    return ok;
}

Sequence *open_mimolix(const Json &config, const std::string &dir, const OpenOptions &opt, std::string &err) {
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
    g.loop_in = g.head && s.loop.times > 0 ? t.matrix("loop.in", s.width, 2 * (size_t)s.width, err) : nullptr;
    if (!g.head || !err.empty() || !t.vector("final.norm", s.width, g.final_norm, err) || !t.vector("final.norm.b", s.width, g.final_bias, err) || model->set_globals(g) != 0)
        return failed();
    return model.release();
}

const RegisterArchitecture kMimolix("Mimolix", open_mimolix);

}  // namespace

}  // namespace bitnet_host
