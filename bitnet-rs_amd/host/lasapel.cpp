// lasapel.cpp -- the Lasapel design: config.json and tensor names -> a StackModel.
//
// Layers of two kinds: attention over a latent (queries through a latent of their own, a learned sink per head, rotary positions
// with YaRN scaling, optionally another layer's cache) and linear attention with constant decays; a dense feed-forward (square of
// relu, biases) or none; norms with weights around zero ahead of and behind every sublayer, a layer scale on what is added.
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
    s.norm_offset = 1.0f;
    const Json *layers = config.find("layers");
    if (!layers || layers->kind != Json::Array || layers->items.empty()) {
        err = "config: layers: missing array";
        return false;
    }
    for (size_t i = 0; i < layers->items.size() && err.empty(); ++i) {
        const JsonView l{&layers->items[i], "layers[" + std::to_string(i) + "].", &err};
        LayerSpec L;
        const std::string type = l.text("type");
        const JsonView m = l.at("mixer");
        if (type == "latent_attention") {
            L.mixer = LayerSpec::Latent;
            LatentSpec &a = L.latent;
            a.heads = m.integer("heads"), a.dim = m.integer("dim"), a.rot_dim = m.integer("rot_dim"), a.vdim = m.integer("vdim");
            a.q_rank = m.integer("q_rank"), a.kv_rank = m.integer("kv_rank");
            a.scale = (float)m.number("scale");
            if (m.has("kv_from")) a.kv_from = m.integer("kv_from", 0);
            const JsonView r = m.at("rot");
            a.rot.dims = r.integer("dims", 2);
            a.rot.base = r.number("base");
            if (r.has("scaling")) {
                const JsonView y = r.at("scaling");
                a.rot.yarn = true;
                a.rot.factor = y.number("factor"), a.rot.original = y.number("original"), a.rot.fast = y.number("fast"), a.rot.slow = y.number("slow");
            }
        } else if (type == "lightning") {
            L.mixer = LayerSpec::Linear;
            L.linear.heads = m.integer("heads"), L.linear.dim = m.integer("dim"), L.linear.vdim = m.integer("vdim");
            L.linear.decay = m.numbers("decay");
        } else if (err.empty()) {
            err = "config: " + l.path + "type: unknown mixer '" + type + "'";
        }
        if (l.has("mlp")) {
            const JsonView f = l.at("mlp");
            if (err.empty() && f.text("kind") != "dense") err = "config: " + f.path + "kind: unknown feed-forward";
            L.ff = f.integer("ff");
            L.act_ff = BITNET_HIP_ACT_RELU2;
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
    bool ok = vec(p + "norm1", w.norm1, W) && vec(p + "norm1b", w.norm1b, W) && vec(p + "ls1", w.ls1, W);
    if (L.mixer == LayerSpec::Latent) {
        const LatentSpec &a = L.latent;
        const size_t H = a.heads;
        ok = ok && mat(m + "dq", &w.dq, a.q_rank, W) && vec(m + "dq.norm", w.dq_norm, a.q_rank) && mat(m + "uq", &w.uq, H * (a.dim + a.rot_dim), a.q_rank) &&
             mat(m + "uk", &w.uk, H * a.dim, a.kv_rank) && mat(m + "uv", &w.uv, H * a.vdim, a.kv_rank) && vec(m + "sink", w.sink, H) &&
             mat(m + "o", &w.o, W, H * a.vdim);
        if (a.kv_from < 0) ok = ok && mat(m + "dkv", &w.dkv, a.kv_rank + a.rot_dim, W) && vec(m + "dkv.norm", w.dkv_norm, a.kv_rank);
    } else {
        const LinearSpec &a = L.linear;
        const size_t H = a.heads;
        ok = ok && mat(m + "q", &w.q, H * a.dim, W) && mat(m + "k", &w.k, H * a.dim, W) && mat(m + "v", &w.v, H * a.vdim, W) && mat(m + "g", &w.g, H * a.vdim, W) &&
             mat(m + "o", &w.o, W, H * a.vdim) && vec(m + "norm", w.out_norm, H * a.vdim);
    }
    if (L.ff > 0)
        ok = ok && vec(p + "norm2", w.norm2, W) && vec(p + "norm2b", w.norm2b, W) && vec(p + "ls2", w.ls2, W) && mat(f + "up", &w.up, L.ff, W) &&
             vec(f + "up.b", w.up_b, L.ff) && mat(f + "down", &w.down, W, L.ff) && vec(f + "down.b", w.down_b, W);
    return ok;
}

Sequence *open_lasapel(const Json &config, const std::string &dir, const OpenOptions &opt, std::string &err) {
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
    if (!g.head || !t.vector("final.norm", s.width, g.final_norm, err) || model->set_globals(g) != 0) return failed();
    return model.release();
}

const RegisterArchitecture kLasapel("Lasapel", open_lasapel);

}  // namespace

}  // namespace bitnet_host
