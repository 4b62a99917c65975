// stack_model.cpp -- see stack_model.hpp.  Host orchestration only: every device operation is a bitnet_hip_* call or plain HIP
// memory plumbing.
#include "stack_model.hpp"

#include <algorithm>
#include <cmath>
#include <cstdio>
#include <cstring>

namespace bitnet_host {

namespace {
constexpr size_t kDecodeSlice = 64;  // queries per call where a portion takes a decode form of its attention
size_t up_to(size_t v, size_t a) { return (v + a - 1) / a * a; }
}  // namespace

std::vector<double> rotary_frequencies(const RotarySpec &r, double *mult) {
    std::vector<double> f((size_t)r.dims / 2);
    for (size_t i = 0; i < f.size(); ++i) f[i] = std::pow(r.base, -2.0 * (double)i / r.dims);
    *mult = 1.0;
    if (r.banded)
        for (double &v : f) {
            const double turns = r.original * v / (2.0 * M_PI), keep = std::min(std::max((turns - r.slow) / (r.fast - r.slow), 0.0), 1.0);
            v = (1.0 - keep) * v / r.factor + keep * v;
        }
    if (!r.yarn) return f;
    // pairs that turn `turns` times within the original length sit at this (fractional) index
    auto index_of = [&](double turns) { return r.dims * std::log(r.original / (2.0 * M_PI * turns)) / (2.0 * std::log(r.base)); };
    const double lo = std::max(std::floor(index_of(r.fast)), 0.0), hi = std::min(std::ceil(index_of(r.slow)), r.dims - 1.0);
    for (size_t i = 0; i < f.size(); ++i) {
        const double ramp = std::min(std::max(((double)i - lo) / std::max(hi - lo, 0.001), 0.0), 1.0);
        f[i] = f[i] / r.factor * ramp + f[i] * (1.0 - ramp);
    }
    *mult = 0.1 * std::log(r.factor) + 1.0;
    return f;
}

StackModel::StackModel(const StackSpec &spec, bool f32, int max_pos) : spec_(spec), f32_(f32), layers_(spec.layers.size()) {
    if (spec.layers.empty() || spec.width <= 0 || spec.vocab <= 0) {
        err_ = "stack: empty model";
        return;
    }
    if (plan_runs() != 0) return;
    for (size_t i = 0; i < layers_.size(); ++i) {
        const LayerSpec &S = spec_.layers[i];
        const bool own = S.mixer == LayerSpec::Attention || S.mixer == LayerSpec::Delta || (S.mixer == LayerSpec::Latent && S.latent.q_rank == 0);
        if ((S.parallel || spec_.residual_gate) && !own) {
            err_ = "stack: layer " + std::to_string(i) + ": side by side with the feed-forward, and gated, stand attention, delta and latent mixers without a query latent only";
            return;
        }
        if (own && plan_block(i, 0, true, S.parallel) != 0) return;
        if (!S.parallel && (S.experts.count > 0 || (spec_.residual_gate && S.ff > 0)) && plan_block(i, 1, false, true) != 0) return;
        if (S.mixer == LayerSpec::Latent && (S.latent.rot_dim != S.latent.rot.dims || S.latent.rot_dim % 2 || S.latent.rot_dim > 256)) {
            err_ = "stack: the rotated part must be even, at most 256 and rotated whole";
            return;
        }
        if ((S.mixer == LayerSpec::Latent || S.mixer == LayerSpec::Attention) && !fits_source(i)) {
            const int from = S.mixer == LayerSpec::Latent ? S.latent.kv_from : S.attention.kv_from;
            err_ = "stack: layer " + std::to_string(i) + " reads the cache of layer " + std::to_string(from) + ", which has none that fits";
            return;
        }
    }
    if (init_sequence(spec.vocab, spec.width, max_pos) != 0) return;
    cap_ = up_to((size_t)max_pos + 1, 128);
    size_t row = 64, eact = 64, z = 64, q = 64, qabs = 64, att = 64, act = 64, lin = 64, lino = 64, scratch = 64;
    const size_t es = f32_ ? 4 : 2;
    for (size_t i = 0; i < layers_.size(); ++i) {
        Layer &L = layers_[i];
        const LayerSpec &S = spec_.layers[i];
        if (S.mixer == LayerSpec::Latent) {
            const LatentSpec &m = S.latent;
            L.dimp = (int)up_to(m.dim, 32), L.rotp = (int)up_to(std::max(m.rot_dim, 1), 32), L.vdimp = (int)up_to(m.vdim, 32), L.ldc = (int)up_to(m.kv_rank, 64);
            if (L.ldc > 1024) {
                err_ = "stack: kv_rank above 1024";
                return;
            }
            z = std::max(z, (size_t)m.q_rank + m.kv_rank + m.rot_dim);
            q = std::max(q, (size_t)m.heads * (L.dimp + L.rotp));
            qabs = std::max(qabs, (size_t)m.heads * L.ldc);
            att = std::max(att, (size_t)m.heads * L.vdimp);
            scratch = std::max(scratch, bitnet_hip_latent_scratch_bytes(m.heads, L.ldc, 1) / 4);
        } else if (S.mixer == LayerSpec::Linear) {
            const LinearSpec &m = S.linear;
            L.dimp = (int)up_to(m.dim, 32), L.vdimp = (int)up_to(m.vdim, 32);
            if (L.dimp > 512 || m.decay.size() != (size_t)m.heads) {
                err_ = "stack: linear attention: head of more than 512 columns, or not one decay per head";
                return;
            }
            lin = std::max(lin, (size_t)m.heads * 2 * (L.dimp + L.vdimp));
            lino = std::max(lino, (size_t)m.heads * L.vdimp);
        } else if (S.mixer == LayerSpec::Attention) {
            scratch = std::max(scratch, bitnet_hip_gqa_scratch_bytes(S.attention.heads, S.attention.maps, L.vdimp, 1) / 4);
        }
        for (const Block &B : L.block)
            if (B.used) {
                row = std::max(row, (size_t)B.ko + B.fs + B.rg + B.main + B.tail);
                eact = std::max(eact, (size_t)S.experts.top * up_to(S.experts.ff, 64));
            }
        act = std::max(act, (size_t)S.ff);
    }
    act = std::max(act, up_to(spec_.side_dim, 8));
    auto vec = [&](float **p, size_t n) { return alloc((void **)p, up_to(n, 64) * 4); };
    bool ok = vec(&x_[0], width_) && vec(&x_[1], width_) && vec(&y_[0], width_) && vec(&y_[1], width_) && vec(&z_, z) && vec(&q_, q) && vec(&qabs_, qabs) &&
              vec(&att_, att) && vec(&act_, act) && vec(&lin_, lin) && vec(&lino_, lino) && vec(&scratch_, scratch) && alloc(&argmax_, 8192) && vec(&x0_, width_) && vec(&row_[0], row) && vec(&row_[1], row) && vec(&h_, width_) && vec(&eact_, eact) &&
              alloc((void **)&eids_, 256);
    for (size_t i = 0; ok && i < layers_.size(); ++i) {
        Layer &L = layers_[i];
        const LayerSpec &S = spec_.layers[i];
        if (S.mixer == LayerSpec::Latent) ok = rope_tables(S.latent.rot, &L.cos, &L.sin) == 0;
        if (S.mixer == LayerSpec::Attention) ok = query_factors(S.attention, &L.q_factor) == 0 && (S.attention.rot.dims == 0 || rope_tables(S.attention.rot, &L.cos, &L.sin) == 0);
        for (Slot &slot : L.slots) {
            if (!ok) break;
            if (S.mixer == LayerSpec::Latent && S.latent.kv_from < 0) {
                ok = alloc(&slot.c, cap_ * L.ldc * es) && alloc(&slot.r, cap_ * L.rotp * es);
            } else if (S.mixer == LayerSpec::Attention) {
                const AttentionSpec &m = S.attention;
                if (m.kv_from < 0) ok = alloc(&slot.k, cap_ * m.kv_heads * m.maps * L.dimp * es) && alloc(&slot.v, cap_ * m.kv_heads * L.vdimp * es);
                if (m.taps > 0) ok = ok && alloc((void **)&slot.ring, (size_t)m.taps * L.channels * 4);
            } else if (S.mixer == LayerSpec::Linear || S.mixer == LayerSpec::Delta) {
                const bool delta = S.mixer == LayerSpec::Delta;
                slot.state_bytes = (size_t)(delta ? S.delta.heads : S.linear.heads) * L.dimp * L.vdimp * 4;
                ok = alloc((void **)&slot.state, slot.state_bytes);
                if (delta) ok = ok && alloc((void **)&slot.ring, (size_t)S.delta.taps * (2 * S.delta.kv_heads * L.dimp + S.delta.heads * L.vdimp) * 4);
            }
        }
    }
    if (!ok) {
        if (err_.empty()) err_ = "device allocation failed";
        return;
    }
    dead_ = false;
    reset();
}

StackModel::~StackModel() {
    drop_graphs();
    for (void *p : owned_) hipFree(p);
    for (Buffer *b : {&px_, &ph_, &pz_, &pcq_, &pq_, &pqf_, &pqabs_, &patt_, &py_, &pact_, &pk_, &pvt_, &plin_, &plinf_, &plino_, &pgate_, &pscratch_, &plws_,
                      &pwant_, &pxw_, &phw_, &plog_, &px0_, &pcat_, &prow_, &ptail_, &pqk_, &pv_, &pgates_, &pplan_, &peact_, &peout_, &pqc_})
        if (b->p) hipFree(b->p);
}

bool StackModel::alloc(void **p, size_t bytes) {
    *p = nullptr;
    if (hipMalloc(p, bytes) != hipSuccess) return false;
    owned_.push_back(*p);
    return hipMemset(*p, 0, bytes) == hipSuccess;
}

// the order in which layers run, and every layer's number of passes
int StackModel::plan_runs() {
    const int n = (int)layers_.size();
    const LoopSpec &loop = spec_.loop;
    if (loop.times != 0 && (loop.times < 1 || loop.start < 0 || loop.stop <= loop.start || loop.stop > n))
        return fail_arg("stack: a loop's range does not lie within the layers");
    for (int i = 0; i < n; ++i) {
        if (loop.times == 0 || i != loop.start) {
            runs_.push_back({(size_t)i, 0, false});
            layers_[(size_t)i].slots.resize(1);
            continue;
        }
        for (int t = 0; t < loop.times; ++t)
            for (int k = loop.start; k < loop.stop; ++k) runs_.push_back({(size_t)k, t, k == loop.start});
        for (int k = loop.start; k < loop.stop; ++k) layers_[(size_t)k].slots.resize((size_t)loop.times);
        i = loop.stop - 1;
    }
    return 0;
}

// a layer that reads the keys and values of an earlier one needs them in its own sizes
bool StackModel::fits_source(size_t i) const {
    const LayerSpec &S = spec_.layers[i];
    const int from = S.mixer == LayerSpec::Latent ? S.latent.kv_from : S.attention.kv_from;
    if (from < 0) return true;
    if ((size_t)from >= i || spec_.layers[(size_t)from].mixer != S.mixer || layers_[(size_t)from].slots.size() != layers_[i].slots.size()) return false;
    if (S.mixer == LayerSpec::Latent) {
        const LatentSpec &a = S.latent, &b = spec_.layers[(size_t)from].latent;
        return b.kv_from < 0 && a.kv_rank == b.kv_rank && a.rot == b.rot && a.neighbours == b.neighbours;
    }
    const AttentionSpec &a = S.attention, &b = spec_.layers[(size_t)from].attention;
    return b.kv_from < 0 && a.kv_heads == b.kv_heads && a.dim == b.dim && a.vdim == b.vdim && a.maps == b.maps && a.rot == b.rot && a.values_are_keys == b.values_are_keys;
}

// sizes of a block and of its mixer's padded heads
int StackModel::plan_block(size_t i, int which, bool mixer, bool ff) {
    Layer &L = layers_[i];
    Block &B = L.block[which];
    const LayerSpec &S = spec_.layers[i];
    const std::string where = "stack: layer " + std::to_string(i) + ": ";
    B.used = true, B.mixer = mixer;
    if (spec_.residual_gate) B.rg = (int)up_to(spec_.width, 64);
    if (mixer && S.mixer == LayerSpec::Attention) {
        const AttentionSpec &m = S.attention;
        L.dimp = (int)up_to(m.dim, 32), L.vdimp = (int)up_to(m.vdim, 32);
        if (m.heads < 1 || m.kv_heads < 1 || m.heads % m.kv_heads || m.maps < 1 || m.maps > 2 || L.dimp > 1024 || L.vdimp > 1024 || !(m.temp_every > 0.0))
            return err_ = where + "attention: query heads in whole groups, one or two maps, heads of up to 1024 columns", BITNET_HIP_ERR_INVALID_ARGUMENT;
        if (m.rot.dims % 2 || m.rot.dims > m.dim || (m.rot.banded && !(m.rot.fast > m.rot.slow)))
            return err_ = where + "attention: an even number of rotated columns within the head, bands in order", BITNET_HIP_ERR_INVALID_ARGUMENT;
        if (m.values_are_keys && (m.vdim != m.dim || m.maps != 1))
            return err_ = where + "attention: keys that are the values have their size, and one map", BITNET_HIP_ERR_INVALID_ARGUMENT;
        if (m.maps != 1 && (m.far_penalty || m.kv_from >= 0 || m.column_gate))
            return err_ = where + "attention: distance penalties, another layer's keys and gates per column go with one map", BITNET_HIP_ERR_INVALID_ARGUMENT;
        if (m.taps < 0 || m.taps > 64 || (m.column_gate && m.head_gate)) return err_ = where + "attention: at most 64 taps, and gates of one kind", BITNET_HIP_ERR_INVALID_ARGUMENT;
        B.ko = (int)up_to((size_t)m.heads * L.vdimp, 64);
        L.channels = L.gate_at = m.kv_from >= 0 ? m.heads * L.dimp : (m.heads + m.kv_heads) * m.maps * L.dimp + (m.values_are_keys ? 0 : m.kv_heads * L.vdimp);
        B.main = L.gate_at + (m.head_gate ? m.heads : m.column_gate ? m.heads * L.vdimp : 0);
    } else if (mixer && S.mixer == LayerSpec::Latent) {
        const LatentSpec &m = S.latent;
        L.dimp = (int)up_to(m.dim, 32), L.rotp = (int)up_to(std::max(m.rot_dim, 1), 32), L.vdimp = (int)up_to(m.vdim, 32);
        B.ko = (int)up_to((size_t)m.heads * L.vdimp, 64);
        B.main = m.heads * (L.dimp + L.rotp);
        B.tail = B.gates = m.kv_from < 0 ? m.kv_rank + m.rot_dim : 0;
    } else if (mixer) {
        const DeltaSpec &m = S.delta;
        L.dimp = (int)up_to(m.dim, 32), L.vdimp = (int)up_to(m.vdim, 32);
        if (m.heads < 1 || m.kv_heads < 1 || m.heads % m.kv_heads || !bitnet_hip_delta_supported(L.dimp, L.vdimp) || m.taps < 1 || m.taps > 64)
            return err_ = where + "delta: value heads in whole groups, heads of up to 256 columns, at most 64 taps", BITNET_HIP_ERR_INVALID_ARGUMENT;
        B.ko = (int)up_to((size_t)m.heads * L.vdimp, 64);
        B.main = 2 * m.kv_heads * L.dimp + 2 * m.heads * L.vdimp;
        B.tail = B.gates = 2 * m.heads;
    }
    if (ff) {
        const ExpertsSpec &e = S.experts;
        B.fs = (int)up_to(S.ff, 64), B.gated = S.gated && S.ff > 0;
        if (S.shared_gate) {
            if (mixer || S.ff == 0 || e.count == 0) return err_ = where + "a gated shared expert stands beside routed ones, behind the mixer", BITNET_HIP_ERR_INVALID_ARGUMENT;
            B.shared = B.tail = B.gates = 1;
        }
        if (e.count > 0) {
            if (e.identity < 0 || e.top < 1 || e.top > e.count + e.identity || e.top > 32 || e.count + e.identity > 1024 || e.ff < 1)
                return err_ = where + "experts: at most 32 of 1024, and not more than there are", BITNET_HIP_ERR_INVALID_ARGUMENT;
            if (e.groups < 0 || (e.groups > 0 && (e.identity > 0 || e.count % e.groups || e.keep < 1 || e.keep > e.groups || e.top > e.keep * (e.count / e.groups))))
                return err_ = where + "experts: equal groups, and enough experts in those that are kept", BITNET_HIP_ERR_INVALID_ARGUMENT;
            B.tail += e.count + e.identity;
        }
    }
    return 0;
}

int StackModel::query_factors(const AttentionSpec &a, float **out) {
    std::vector<float> f(cap_);
    for (size_t p = 0; p < cap_; ++p) f[p] = (float)(a.scale * (1.0 + a.temp_coef * std::log(std::floor((double)(p + 1) / a.temp_every) + 1.0)));
    return upload(out, f);
}

int StackModel::grow(Buffer &b, size_t bytes) {
    if (b.bytes >= bytes) return 0;
    if (b.p) {
        HCHK(hipStreamSynchronize((hipStream_t)stream_));
        HCHK(hipFree(b.p));
    }
    b.p = nullptr;
    b.bytes = 0;
    HCHK(hipMalloc(&b.p, bytes));
    HCHK(hipMemset(b.p, 0, bytes));
    HCHK(hipDeviceSynchronize());
    b.bytes = bytes;
    return 0;
}

template <class T>
int StackModel::upload(T **dst, const std::vector<T> &src) {
    *dst = nullptr;
    if (src.empty()) return 0;
    void *p = nullptr;
    const size_t bytes = up_to(src.size() * sizeof(T), 256);
    HCHK(hipMalloc(&p, bytes));
    owned_.push_back(p);
    HCHK(hipMemset(p, 0, bytes));
    HCHK(hipMemcpy(p, src.data(), src.size() * sizeof(T), hipMemcpyHostToDevice));
    *dst = static_cast<T *>(p);
    return 0;
}

// dense rows [n_rows][cols] -> the device layout
int StackModel::upload_matrix(Matrix &m, const std::vector<uint16_t> &rows, int n_rows, int cols) {
    m.rows = n_rows, m.cols = (int)up_to(cols, 8), m.ld = (int)up_to(cols, 64);
    void *p = nullptr;
    HCHK(hipMalloc(&p, (size_t)n_rows * m.ld * 2));
    owned_.push_back(p);
    HCHK(hipMemset(p, 0, (size_t)n_rows * m.ld * 2));
    HCHK(hipMemcpy2D(p, (size_t)m.ld * 2, rows.data(), (size_t)cols * 2, (size_t)cols * 2, n_rows, hipMemcpyHostToDevice));
    m.w = static_cast<uint16_t *>(p);
    weight_bytes_ += (size_t)n_rows * cols * 2;
    return 0;
}

int StackModel::rope_tables(const RotarySpec &r, float **cos, float **sin) {
    for (const RopeTable &t : ropes_)
        if (t.spec == r) return *cos = t.cos, *sin = t.sin, 0;
    double mult = 1.0;
    const std::vector<double> f = rotary_frequencies(r, &mult);
    std::vector<float> c(cap_ * f.size()), s(cap_ * f.size());
    for (size_t p = 0; p < cap_; ++p)
        for (size_t i = 0; i < f.size(); ++i) {
            const double a = (double)p * f[i];
            c[p * f.size() + i] = (float)(std::cos(a) * mult);
            s[p * f.size() + i] = (float)(std::sin(a) * mult);
        }
    if (c.empty()) c.resize(1), s.resize(1);
    if (int rc = upload(cos, c)) return rc;
    if (int rc = upload(sin, s)) return rc;
    ropes_.push_back({r, *cos, *sin});
    return 0;
}

// ---- weights ----------------------------------------------------------------------------------------------------------

namespace {
// rows [groups][from] of a matrix with `cols` columns -> [groups][to], the new rows zero
std::vector<uint16_t> pad_rows(const uint16_t *w, size_t groups, size_t from, size_t to, size_t cols) {
    std::vector<uint16_t> o(groups * to * cols, 0);
    for (size_t g = 0; g < groups; ++g) memcpy(&o[g * to * cols], w + g * from * cols, from * cols * 2);
    return o;
}
// columns [groups][from] -> [groups][to]
std::vector<uint16_t> pad_cols(const uint16_t *w, size_t rows, size_t groups, size_t from, size_t to) {
    std::vector<uint16_t> o(rows * groups * to, 0);
    for (size_t r = 0; r < rows; ++r)
        for (size_t g = 0; g < groups; ++g) memcpy(&o[(r * groups + g) * to], w + (r * groups + g) * from, from * 2);
    return o;
}
// short convolution weights [groups][from channels][taps] into rows [taps][channels] at column `at`
void put_taps(std::vector<float> &rows, size_t channels, size_t at, const std::vector<float> &w, size_t groups, size_t from, size_t to, size_t taps) {
    for (size_t g = 0; g < groups; ++g)
        for (size_t c = 0; c < from; ++c)
            for (size_t j = 0; j < taps; ++j) rows[j * channels + at + g * to + c] = w[(g * from + c) * taps + j];
}
// a vector [groups][from] at `at` of another one, [groups][to]
void put_heads(std::vector<float> &o, size_t at, const std::vector<float> &v, size_t groups, size_t from, size_t to) {
    for (size_t g = 0; g < groups; ++g) std::copy(v.begin() + g * from, v.begin() + (g + 1) * from, o.begin() + at + g * to);
}
// where the j-th row of a rotated part of n rows comes from: pairs of neighbours lie half of the part apart on the device
size_t rotated_row(bool neighbours, size_t n, size_t j) { return !neighbours ? j : j < n / 2 ? 2 * j : 2 * (j - n / 2) + 1; }
// rows of two matrices in turn
void append_pairs(std::vector<uint16_t> &o, const uint16_t *a, const uint16_t *b, size_t rows, size_t cols) {
    for (size_t r = 0; r < rows; ++r) {
        o.insert(o.end(), a + r * cols, a + (r + 1) * cols);
        o.insert(o.end(), b + r * cols, b + (r + 1) * cols);
    }
}
double dot(const std::vector<float> &a, const std::vector<float> &b) {
    double s = 0.0;
    for (size_t i = 0; i < a.size(); ++i) s += (double)a[i] * b[i];
    return s;
}
std::vector<uint16_t> take(const uint16_t *w, size_t n) { return std::vector<uint16_t>(w, w + n); }
void append(std::vector<uint16_t> &a, const std::vector<uint16_t> &b) { a.insert(a.end(), b.begin(), b.end()); }
}  // namespace

#define TRY(expr)                \
    do {                         \
        if (int _r = (expr)) return _r; \
    } while (0)

int StackModel::set_layer(int layer, const StackLayerWeights &w) {
    if (layer < 0 || (size_t)layer >= layers_.size()) return fail_arg("layer index out of range");
    Layer &L = layers_[(size_t)layer];
    const LayerSpec &S = spec_.layers[(size_t)layer];
    const size_t W = width_;
    if (L.set) return fail_arg("the layer already holds weights");
    auto sized = [&](const std::vector<float> &v) { return v.empty() || v.size() == W; };
    if (!sized(w.norm1) || !sized(w.norm1b) || !sized(w.ls1) || !sized(w.norm1_bias) || (!w.ls1.empty() && w.norm1b.empty()))
        return fail_arg("stack: norm of the wrong size");
    const size_t before = weight_bytes_;
    TRY(upload(&L.norm1.w, w.norm1));
    TRY(upload(&L.norm1.bias, w.norm1_bias));
    TRY(upload(&L.norm1b, w.norm1b));
    TRY(upload(&L.ls1, w.ls1));
    L.act_a = w.act_a, L.act_b = w.act_b;
    if (S.mixer == LayerSpec::Latent && S.latent.q_rank > 0) {
        const LatentSpec &m = S.latent;
        const size_t H = m.heads, D = m.dim, R = m.rot_dim, V = m.vdim;
        if (m.neighbours) return fail_arg("stack: neighbours turn together in queries straight from the input only");
        if (!w.dq || !w.uq || !w.uk || !w.uv || !w.o || (m.kv_from < 0) != (w.dkv != nullptr) || w.dq_norm.size() != (size_t)m.q_rank || w.sink.size() != H ||
            (m.kv_from < 0 && w.dkv_norm.size() != (size_t)m.kv_rank))
            return fail_arg("stack: incomplete latent attention weights");
        std::vector<uint16_t> t = take(w.dq, m.q_rank * W);
        if (w.dkv) append(t, take(w.dkv, (m.kv_rank + R) * W));
        TRY(upload_matrix(L.down_q, t, (int)(t.size() / W), (int)W));
        // queries: every head's unrotated part, then its rotated part, each padded on its own
        const size_t qd = L.dimp + L.rotp;
        t.assign(H * qd * m.q_rank, 0);
        for (size_t h = 0; h < H; ++h) {
            memcpy(&t[h * qd * m.q_rank], w.uq + h * (D + R) * m.q_rank, D * m.q_rank * 2);
            memcpy(&t[(h * qd + L.dimp) * m.q_rank], w.uq + (h * (D + R) + D) * m.q_rank, R * m.q_rank * 2);
        }
        TRY(upload_matrix(L.uq, t, (int)(H * qd), m.q_rank));
        TRY(set_latent(L, m, w));
        TRY(upload_matrix(L.o, pad_cols(w.o, W, H, V, L.vdimp), (int)W, (int)(H * L.vdimp)));
        TRY(upload(&L.dq_norm, w.dq_norm));
    } else if (S.mixer == LayerSpec::Linear) {
        const LinearSpec &m = S.linear;
        const size_t H = m.heads, D = m.dim, V = m.vdim;
        if (!w.q || !w.k || !w.v || !w.g || !w.o || w.out_norm.size() != H * V) return fail_arg("stack: incomplete linear attention weights");
        std::vector<uint16_t> t = pad_rows(w.q, H, D, L.dimp, W);
        append(t, pad_rows(w.k, H, D, L.dimp, W));
        append(t, pad_rows(w.v, H, V, L.vdimp, W));
        append(t, pad_rows(w.g, H, V, L.vdimp, W));
        TRY(upload_matrix(L.qkvg, t, (int)(H * 2 * (L.dimp + L.vdimp)), (int)W));
        TRY(upload_matrix(L.o, pad_cols(w.o, W, H, V, L.vdimp), (int)W, (int)(H * L.vdimp)));
        std::vector<float> n(H * L.vdimp, 0.f), pw(H * (BITNET_HIP_LINEAR_BLOCK + 1));
        for (size_t h = 0; h < H; ++h) {
            for (size_t v = 0; v < V; ++v) n[h * L.vdimp + v] = w.out_norm[h * V + v];
            double p = 1.0;
            for (size_t i = 0; i <= BITNET_HIP_LINEAR_BLOCK; ++i, p *= m.decay[h]) pw[h * (BITNET_HIP_LINEAR_BLOCK + 1) + i] = (float)p;
        }
        TRY(upload(&L.out_norm, n));
        TRY(upload(&L.decay_pow, pw));
    }
    if (!S.parallel && (S.ff > 0 || S.experts.count > 0)) {
        if (!sized(w.norm2) || !sized(w.norm2b) || !sized(w.ls2) || !sized(w.norm2_bias) || (!w.ls2.empty() && w.norm2b.empty()))
            return fail_arg("stack: norm of the wrong size");
        TRY(upload(&L.norm2.w, w.norm2));
        TRY(upload(&L.norm2.bias, w.norm2_bias));
        TRY(upload(&L.norm2b, w.norm2b));
        TRY(upload(&L.ls2, w.ls2));
    }
    for (int b = 0; b < 2; ++b)
        if (L.block[b].used) TRY(set_block((size_t)layer, b, w));
    if (spec_.side_dim > 0) {
        if (!w.side_gate || !w.side_proj || w.side_norm.size() != W) return fail_arg("stack: incomplete token input");
        TRY(upload_matrix(L.side_gate, take(w.side_gate, (size_t)spec_.side_dim * W), spec_.side_dim, (int)W));
        TRY(upload_matrix(L.side_proj, take(w.side_proj, W * spec_.side_dim), (int)W, spec_.side_dim));
        std::vector<float> norm = w.side_norm;  // (a plain weight, whatever the model's norms have)
        for (float &v : norm) v -= spec_.norm_offset;
        TRY(upload(&L.side_norm, norm));
    }
    if (!S.parallel && S.ff > 0 && S.experts.count == 0 && !L.block[1].used) {
        const size_t F = S.ff;
        if (!w.up || !w.down || S.gated != (w.gate != nullptr) || (!w.up_b.empty() && (S.gated || w.up_b.size() != F)) || (!w.down_b.empty() && w.down_b.size() != W))
            return fail_arg("stack: incomplete feed-forward weights");
        if (S.gated) {
            std::vector<uint16_t> t;
            append_pairs(t, w.gate, w.up, F, W);
            TRY(upload_matrix(L.up, t, (int)(2 * F), (int)W));
        } else {
            TRY(upload_matrix(L.up, take(w.up, F * W), (int)F, (int)W));
        }
        TRY(upload_matrix(L.down, take(w.down, W * F), (int)W, (int)F));
        TRY(upload(&L.up_b, w.up_b));
        TRY(upload(&L.down_b, w.down_b));
    }
    weight_bytes_ = before + (weight_bytes_ - before) * L.slots.size();  // every pass reads them
    L.set = true;
    ++layers_set_;
    return 0;
}

// what latent attention needs besides its down-projections and its output
int StackModel::set_latent(Layer &L, const LatentSpec &m, const StackLayerWeights &w) {
    const size_t H = m.heads, D = m.dim, V = m.vdim;
    // W_uk twice: as it is (the prompt expands keys) and per head transposed (a step takes the query into latent space)
    TRY(upload_matrix(L.uk, pad_rows(w.uk, H, D, L.dimp, m.kv_rank), (int)(H * L.dimp), m.kv_rank));
    std::vector<uint16_t> t(H * L.ldc * L.dimp, 0);
    for (size_t h = 0; h < H; ++h)
        for (size_t d = 0; d < D; ++d)
            for (size_t c = 0; c < (size_t)m.kv_rank; ++c) t[(h * L.ldc + c) * L.dimp + d] = w.uk[(h * D + d) * m.kv_rank + c];
    TRY(upload_matrix(L.uk_t, t, (int)(H * L.ldc), L.dimp));
    weight_bytes_ -= t.size() * 2;  // one of the two copies is read per token
    TRY(upload_matrix(L.uv, pad_rows(w.uv, H, V, L.vdimp, m.kv_rank), (int)(H * L.vdimp), m.kv_rank));
    TRY(upload(&L.dkv_norm, w.dkv_norm));
    return upload(&L.sink, w.sink);
}

int StackModel::set_block(size_t i, int which, const StackLayerWeights &w) {
    Layer &L = layers_[i];
    Block &B = L.block[which];
    const LayerSpec &S = spec_.layers[i];
    const size_t W = width_, F = B.mixer && !S.parallel ? 0 : S.ff;
    const ExpertsSpec E = B.mixer && !S.parallel ? ExpertsSpec() : S.experts;
    B.norm = which == 0 ? L.norm1 : L.norm2;
    std::vector<uint16_t> in, out(W * (B.ko + B.fs), 0);
    std::vector<float> bias((size_t)B.ff_rows() + B.rg + B.main + B.tail, 0.f);
    bool biased = false;
    auto put_bias = [&](size_t at, const std::vector<float> &v, size_t groups, size_t from, size_t to) {
        if (!v.empty()) put_heads(bias, at, v, groups, from, to), biased = true;
    };
    auto into_out = [&](const uint16_t *m, size_t at, size_t groups, size_t from, size_t to) {
        for (size_t r = 0; r < W; ++r)
            for (size_t g = 0; g < groups; ++g) memcpy(&out[r * (B.ko + B.fs) + at + g * to], m + (r * groups + g) * from, from * 2);
    };
    if (F > 0) {
        if (!w.up || !w.down || B.gated != (w.gate != nullptr) || (!w.up_b.empty() && (B.gated || w.up_b.size() != F)) || (!w.down_b.empty() && w.down_b.size() != W) ||
            (B.shared != 0) != (w.shared_gate != nullptr))
            return fail_arg("stack: incomplete feed-forward weights");
        if (B.gated)
            append_pairs(in, w.gate, w.up, F, W);
        else
            append(in, take(w.up, F * W));
        in.resize((size_t)B.ff_rows() * W, 0);
        put_bias(0, w.up_b, 1, F, F);
        into_out(w.down, B.ko, 1, F, F);
    }
    if (B.rg > 0) {
        const uint16_t *m = which == 0 ? w.rg1 : w.rg2;
        const std::vector<float> &b = which == 0 ? w.rg1_b : w.rg2_b;
        if (!m || (!b.empty() && b.size() != W)) return fail_arg("stack: incomplete residual gate");
        append(in, take(m, W * W));
        in.resize((size_t)(B.ff_rows() + B.rg) * W, 0);
        put_bias(B.ff_rows(), b, 1, W, W);
    }
    const size_t proj = B.ff_rows() + B.rg;  // rows ahead of the mixer's
    if (B.mixer && S.mixer == LayerSpec::Attention) {
        const AttentionSpec &m = S.attention;
        const size_t H = m.heads, G = m.kv_heads, M = m.maps, D = m.dim, V = m.vdim;
        const bool two = M == 2 && w.lq1.size() == D && w.lk1.size() == D && w.lq2.size() == D && w.lk2.size() == D;
        const bool owns = m.kv_from < 0, values = owns && !m.values_are_keys;
        auto sized = [](const std::vector<float> &v, size_t n) { return v.empty() || v.size() == n; };
        if (!w.q || owns != (w.k != nullptr) || values != (w.v != nullptr) || (m.head_gate || m.column_gate) != (w.g != nullptr) || !w.o || !sized(w.q_norm, D) ||
            !sized(w.k_norm, D) || (M == 2 && !two) || (!w.sink.empty() && (w.sink.size() != H || M == 2)) || !sized(w.q_b, H * M * D) || !sized(w.k_b, owns ? G * M * D : 0) ||
            !sized(w.v_b, values ? G * V : 0) || (m.far_penalty && (w.far_weight.size() != H || w.far_rate.size() != H)))
            return fail_arg("stack: incomplete attention weights");
        append(in, pad_rows(w.q, H * M, D, L.dimp, W));
        if (w.k) append(in, pad_rows(w.k, G * M, D, L.dimp, W));
        if (w.v) append(in, pad_rows(w.v, G, V, L.vdimp, W));
        if (w.g) append(in, m.column_gate ? pad_rows(w.g, H, V, L.vdimp, W) : take(w.g, H * W));
        const size_t k_at = H * M * L.dimp, v_at = k_at + G * M * L.dimp;
        put_bias(proj, w.q_b, H * M, D, L.dimp);
        put_bias(proj + k_at, w.k_b, G * M, D, L.dimp);
        put_bias(proj + v_at, w.v_b, G, V, L.vdimp);
        if (m.taps > 0) {
            const size_t T = m.taps, C = L.channels;
            if (w.q_conv.size() != H * M * D * T || w.k_conv.size() != (owns ? G * M * D * T : 0) || w.v_conv.size() != (values ? G * V * T : 0))
                return fail_arg("stack: incomplete convolutions");
            std::vector<float> conv(T * C, 0.f);
            put_taps(conv, C, 0, w.q_conv, H * M, D, L.dimp, T);
            if (owns) put_taps(conv, C, k_at, w.k_conv, G * M, D, L.dimp, T);
            if (values) put_taps(conv, C, v_at, w.v_conv, G, V, L.vdimp, T);
            TRY(upload(&L.conv, conv));
        }
        if (m.far_penalty) {
            TRY(upload(&L.far_weight, w.far_weight));
            TRY(upload(&L.far_rate, w.far_rate));
        }
        into_out(w.o, 0, H, V, L.vdimp);
        TRY(upload(&L.sink, w.sink));
        TRY(upload(&L.q_norm, w.q_norm));
        TRY(upload(&L.k_norm, w.k_norm));
        if (two) L.lambda = (float)(std::exp(dot(w.lq1, w.lk1)) - std::exp(dot(w.lq2, w.lk2)) + m.diff);
    } else if (B.mixer && S.mixer == LayerSpec::Latent) {
        const LatentSpec &m = S.latent;
        const size_t H = m.heads, D = m.dim, R = m.rot_dim, V = m.vdim, qd = L.dimp + L.rotp;
        if (!w.q || !w.uk || !w.uv || !w.o || (m.kv_from < 0) != (w.dkv != nullptr) || (!w.sink.empty() && w.sink.size() != H) ||
            (m.kv_from < 0 && w.dkv_norm.size() != (size_t)m.kv_rank))
            return fail_arg("stack: incomplete latent attention weights");
        // every head's unrotated part, then its rotated part, each padded on its own
        std::vector<uint16_t> t(H * qd * W, 0);
        for (size_t h = 0; h < H; ++h) {
            memcpy(&t[h * qd * W], w.q + h * (D + R) * W, D * W * 2);
            for (size_t j = 0; j < R; ++j) memcpy(&t[(h * qd + L.dimp + j) * W], w.q + (h * (D + R) + D + rotated_row(m.neighbours, R, j)) * W, W * 2);
        }
        append(in, t);
        if (w.dkv) {
            append(in, take(w.dkv, m.kv_rank * W));
            for (size_t j = 0; j < R; ++j) append(in, take(w.dkv + (m.kv_rank + rotated_row(m.neighbours, R, j)) * W, W));
        }
        into_out(w.o, 0, H, V, L.vdimp);
        TRY(set_latent(L, m, w));
    } else if (B.mixer) {
        const DeltaSpec &m = S.delta;
        const size_t H = m.heads, G = m.kv_heads, D = m.dim, V = m.vdim, T = m.taps, C = 2 * G * L.dimp + H * L.vdimp;
        if (!w.q || !w.k || !w.v || !w.g || !w.o || !w.b || !w.a || w.q_conv.size() != G * D * T || w.k_conv.size() != G * D * T || w.v_conv.size() != H * V * T ||
            w.a_log.size() != H || w.dt_bias.size() != H || w.out_norm.size() != V)
            return fail_arg("stack: incomplete delta weights");
        append(in, pad_rows(w.q, G, D, L.dimp, W));
        append(in, pad_rows(w.k, G, D, L.dimp, W));
        append(in, pad_rows(w.v, H, V, L.vdimp, W));
        append(in, pad_rows(w.g, H, V, L.vdimp, W));
        append(in, take(w.b, H * W));
        append(in, take(w.a, H * W));
        into_out(w.o, 0, H, V, L.vdimp);
        std::vector<float> conv(T * C, 0.f), rate(H), norm(L.vdimp, 0.f);
        put_taps(conv, C, 0, w.q_conv, G, D, L.dimp, T);
        put_taps(conv, C, G * L.dimp, w.k_conv, G, D, L.dimp, T);
        put_taps(conv, C, 2 * G * L.dimp, w.v_conv, H, V, L.vdimp, T);
        for (size_t h = 0; h < H; ++h) rate[h] = (float)std::exp((double)w.a_log[h]);
        std::copy(w.out_norm.begin(), w.out_norm.end(), norm.begin());
        TRY(upload(&L.conv, conv));
        TRY(upload(&L.decay_rate, rate));
        TRY(upload(&L.dt_bias, w.dt_bias));
        TRY(upload(&L.out_norm, norm));
    }
    if (E.count > 0) {
        const size_t N = E.count, R = E.ff;
        const size_t outputs = N + E.identity, up_rows = E.gated ? 2 * R : R;
        if (!w.router || w.expert_up.size() != N || w.expert_down.size() != N || w.expert_gate.size() != (E.gated ? N : 0) ||
            (!w.router_correction.empty() && w.router_correction.size() != outputs))
            return fail_arg("stack: incomplete experts");
        if (B.shared) append(in, take(w.shared_gate, W));
        append(in, take(w.router, outputs * W));
        TRY(upload(&L.correction, w.router_correction));
        std::vector<uint16_t> up, down;
        for (size_t e = 0; e < N; ++e) {
            if (!w.expert_up[e] || !w.expert_down[e] || (E.gated && !w.expert_gate[e])) return fail_arg("stack: incomplete experts");
            if (E.gated)
                append_pairs(up, w.expert_gate[e], w.expert_up[e], R, W);
            else
                up.insert(up.end(), w.expert_up[e], w.expert_up[e] + R * W);
            down.insert(down.end(), w.expert_down[e], w.expert_down[e] + W * R);
        }
        TRY(upload_matrix(B.expert_up, up, (int)(N * up_rows), (int)W));
        TRY(upload_matrix(B.expert_down, down, (int)(N * W), (int)R));
        weight_bytes_ -= (N - std::min(N, (size_t)E.top)) * (up_rows + R) * W * 2;  // a token reads `top` of them (fewer where identities are chosen)
    }
    if (in.size() != bias.size() * W) return fail_arg("stack: a block's rows do not add up");
    TRY(upload_matrix(B.in, in, (int)bias.size(), (int)W));
    if (B.ko + B.fs > 0) TRY(upload_matrix(B.out, out, (int)W, B.ko + B.fs));
    if (biased) TRY(upload(&B.in_bias, bias));
    if (F > 0) TRY(upload(&B.out_bias, w.down_b));
    return 0;
}

int StackModel::set_globals(const StackGlobalWeights &w) {
    const size_t W = width_;
    if (!w.embed || (!w.embed_norm.empty() && w.embed_norm.size() != W) || w.final_norm.size() != W || (!w.final_bias.empty() && w.final_bias.size() != W) || !w.head ||
        (spec_.loop.times > 0) != (w.loop_in != nullptr) || (spec_.pairs.buckets > 0) != (w.pairs != nullptr) || (spec_.side_dim > 0) != (w.side != nullptr) ||
        (w.pairs && !w.embed_norm.empty()))
        return fail_arg("stack: incomplete globals");
    if (head_) return fail_arg("the model already holds its globals");
    const size_t n = (size_t)vocab_ * W;
    const size_t before = weight_bytes_;
    TRY(upload_matrix(embed_, take(w.embed, n), vocab_, width_));
    if (w.pairs) TRY(upload_matrix(pairs_, take(w.pairs, (spec_.pairs.buckets + 1) * W), (int)spec_.pairs.buckets + 1, width_));
    if (w.side) {
        const size_t cols = layers_.size() * (size_t)spec_.side_dim;
        TRY(upload_matrix(side_, take(w.side, vocab_ * cols), vocab_, (int)cols));
    }
    weight_bytes_ = before;  // a row of each is read per token
    TRY(upload_matrix(head_m_, take(w.head, n), vocab_, width_));
    TRY(upload(&embed_norm_, w.embed_norm));
    TRY(upload(&final_norm_.w, w.final_norm));
    TRY(upload(&final_norm_.bias, w.final_bias));
    if (w.loop_in) {
        TRY(upload_matrix(loop_in_, take(w.loop_in, 2 * W * W), width_, 2 * width_));
        weight_bytes_ += (size_t)(spec_.loop.times - 1) * 4 * W * W;
    }
    head_ = head_m_.w;
    return 0;
}

int StackModel::clear_state() {
    // the caches need no clearing: a position is read only after it was written, what lies past it meets a zero weight
    // (a convolution's earlier inputs are read for positions of this sequence only)
    for (const Layer &L : layers_)
        for (const Slot &slot : L.slots)
            if (slot.state) HCHK(hipMemsetAsync(slot.state, 0, slot.state_bytes, (hipStream_t)stream_));
    HCHK(hipStreamSynchronize((hipStream_t)stream_));
    hidden_ = nullptr;
    return 0;
}

// proj: rows of projections (the heads' gates stay in them)
bitnet_hip_gqa StackModel::gqa_args(size_t i, int pass, const void *proj, size_t ld, bool f32) const {
    const Layer &L = layers_[i];
    const AttentionSpec &m = spec_.layers[i].attention;
    const Slot &slot = kv_slot(i, pass);
    bitnet_hip_gqa a;
    memset(&a, 0, sizeof(a));
    a.heads = m.heads, a.kv_heads = m.kv_heads, a.maps = m.maps, a.dim = m.dim, a.dimp = L.dimp, a.vdim = m.vdim, a.vdimp = L.vdimp, a.capacity = cap_;
    a.eps = spec_.eps, a.lambda = L.lambda, a.out_scale = 1.0f - m.diff, a.q_weight = L.q_norm, a.k_weight = L.k_norm, a.q_factor = L.q_factor;
    a.kcache = slot.k, a.vcache = slot.v;
    a.unit_norm = m.unit_norm, a.values_are_keys = m.values_are_keys, a.rot_dims = m.rot.dims, a.chunk = m.chunk, a.rope_cos = L.cos, a.rope_sin = L.sin, a.sink = L.sink;
    a.window = m.window, a.queries_only = m.kv_from >= 0, a.far_weight = L.far_weight, a.far_rate = L.far_rate, a.gate_columns = m.column_gate;
    if (m.head_gate || m.column_gate) a.gate = (const char *)proj + (size_t)L.gate_at * (f32 ? 4 : 2), a.ldgate = ld, a.gate_f32 = f32;
    return a;
}

bitnet_hip_router StackModel::router_args(size_t i) const {
    const ExpertsSpec &e = spec_.layers[i].experts;
    bitnet_hip_router r;
    memset(&r, 0, sizeof(r));
    r.experts = e.count, r.identity = e.identity, r.top = e.top, r.scale = e.scale, r.raw = e.raw, r.correction = layers_[i].correction;
    r.sigmoid = e.sigmoid, r.groups = e.groups, r.keep = e.keep;
    return r;
}

bitnet_hip_delta StackModel::delta_args(size_t i, int pass) const {
    const Layer &L = layers_[i];
    const DeltaSpec &m = spec_.layers[i].delta;
    const Slot &slot = L.slots[(size_t)pass];
    bitnet_hip_delta d;
    memset(&d, 0, sizeof(d));
    d.heads = m.heads, d.kv_heads = m.kv_heads, d.dim = m.dim, d.dimp = L.dimp, d.vdim = m.vdim, d.vdimp = L.vdimp, d.taps = m.taps;
    d.conv = L.conv, d.decay_rate = L.decay_rate, d.dt_bias = L.dt_bias, d.norm = L.out_norm;
    d.q_scale = (float)(1.0 / std::sqrt((double)m.dim)), d.unit_eps = m.unit_eps, d.eps = spec_.eps, d.state = slot.state, d.ring = slot.ring;
    return d;
}

void StackModel::attention_args(size_t i, int pass, bitnet_hip_latent_attention &a) const {
    const Layer &L = layers_[i];
    const Slot &K = kv_slot(i, pass);
    const LatentSpec &m = spec_.layers[i].latent;
    a.heads = m.heads, a.dimp = L.dimp, a.qd = L.dimp + L.rotp, a.vdimp = L.vdimp, a.kv_rank = m.kv_rank, a.rot_dim = m.rot_dim;
    a.scale = m.scale, a.sink = L.sink, a.ccache = K.c, a.rcache = K.r, a.ldc = L.ldc, a.ldr = L.rotp, a.capacity = cap_;
    a.rope_cos = L.cos, a.rope_sin = L.sin, a.ldq = 0;
}

void StackModel::latent_args(size_t i, int pass, const float *z, size_t ldz, void *cq, size_t ldcq, bitnet_hip_latent_rows &r) const {
    const Layer &L = layers_[i];
    const LatentSpec &m = spec_.layers[i].latent;
    memset(&r, 0, sizeof(r));
    r.z = z, r.ldz = ldz, r.q_rank = m.q_rank, r.q_weight = L.dq_norm, r.eps = spec_.eps, r.cq = cq, r.ldcq = ldcq, r.pos = pos_;
    if (m.kv_from < 0) {
        r.kv_rank = m.kv_rank, r.rot_dim = m.rot_dim, r.kv_weight = L.dkv_norm;
        r.ccache = L.slots[(size_t)pass].c, r.rcache = L.slots[(size_t)pass].r, r.ldc = L.ldc, r.ldr = L.rotp, r.rope_cos = L.cos, r.rope_sin = L.sin;
    }
}

// ---- one token --------------------------------------------------------------------------------------------------------
// *cur_ is the residual stream up to the pending sublayer; the launch that normalises it for the next sublayer adds the pending
// output on the way and leaves the sum in another buffer.

int StackModel::gemv(const bitnet_hip_vector_input &in, const Matrix &m, const float *bias, int act0, int act1, size_t split, float *y,
                     const bitnet_hip_latent_rows *latent, const bitnet_hip_epilogue *more) {
    BCHK(bitnet_hip_dense_gemv_dev(&in, m.w, m.rows, m.cols, m.ld, bias, act0, act1, split, y, 1, 0, 0, 0, latent, f32_, more, stream_));
    return 0;
}

static bitnet_hip_vector_input plain_input(const float *x) {
    bitnet_hip_vector_input in;
    memset(&in, 0, sizeof(in));
    in.x = x;
    in.kind = BITNET_HIP_IN_PLAIN;
    return in;
}

void StackModel::add_pending(bitnet_hip_vector_input &in) {
    if (!pending_.y) return;
    cur_ = in.x_out = next_x();
    in.y = pending_.y, in.post_weight = pending_.w, in.scale = pending_.scale, in.mult = spec_.residual_mult, in.y_gate = (const float *)pending_.gate;
    pending_ = Pending();
}

bitnet_hip_vector_input StackModel::block_input(const Norm &norm) {
    bitnet_hip_vector_input in = plain_input(cur_);
    in.kind = norm.w ? BITNET_HIP_IN_RESIDUAL_NORM : BITNET_HIP_IN_RESIDUAL;
    in.eps = spec_.eps, in.weight_offset = spec_.norm_offset, in.weight = norm.w, in.bias = norm.bias, in.center = spec_.center, in.n = width_;
    add_pending(in);
    return in;
}

// x <- W_in [x; embedding output]
int StackModel::step_loop_in() {
    bitnet_hip_vector_input in = plain_input(cur_);
    in.kind = BITNET_HIP_IN_CONCAT, in.n = width_, in.x2 = x0_;
    add_pending(in);
    in.x_out = nullptr;  // (nobody else reads the sum)
    float *x = in.x == x_[0] ? x_[1] : x_[0];
    TRY(gemv(in, loop_in_, nullptr, 0, 0, 0, x));
    cur_ = x;
    return 0;
}

// the sublayers of a block; their sum is left in y_[which]
int StackModel::step_block(size_t i, int pass, int which) {
    const Layer &L = layers_[i];
    const Block &B = L.block[which];
    const LayerSpec &S = spec_.layers[i];
    const bool routed = B.expert_up.w != nullptr;
    bitnet_hip_vector_input in = block_input(B.norm);
    const float *h = B.norm.w ? h_ : cur_;  // what the experts read
    if (routed && B.norm.w) in.h_out = h_;
    row_at_ ^= 1;
    float *row = row_[row_at_], *proj = row + B.ko + B.fs + B.rg, *tail = proj + B.main;
    // feed-forward | residual gate and the shared expert's number | the rest
    bitnet_hip_epilogue more = {};
    const int gates = B.rg + B.shared, gate_act = gates ? BITNET_HIP_ACT_SIGMOID : 0;
    more.act_a = L.act_a, more.act_b = L.act_b;
    if (B.gated) more.pairs = B.ff_rows();
    if (B.fs && gates) more.act2_from = B.ff_rows() + gates;
    if (B.mixer && S.mixer == LayerSpec::Attention && S.attention.taps > 0) {
        more.conv_from = B.ff_rows() + B.rg, more.channels = L.channels, more.taps = S.attention.taps;
        more.conv = L.conv, more.ring = L.slots[(size_t)pass].ring, more.pos = pos_;
    }
    if (B.fs)
        TRY(gemv(in, B.in, B.in_bias, S.act_ff | (B.gated ? BITNET_HIP_ACT_GATED : 0), gate_act, B.ff_rows(), row + B.ko, nullptr, &more));
    else
        TRY(gemv(in, B.in, B.in_bias, gate_act, 0, gates, row + B.ko, nullptr, &more));
    if (B.mixer && S.mixer == LayerSpec::Latent) {
        bitnet_hip_latent_rows r;
        latent_args(i, pass, tail, B.tail, nullptr, 0, r);
        TRY(step_attend_latent(i, pass, proj, S.latent.kv_from < 0 ? &r : nullptr, row, B.ko));
    } else if (B.mixer && S.mixer == LayerSpec::Attention) {
        const bitnet_hip_gqa a = gqa_args(i, pass, proj, B.main, true);
        if (!f32_ && bitnet_hip_gqa_supported(a.dimp, a.vdimp)) {
            BCHK(bitnet_hip_gqa_step_dev(&a, proj, pos_, scratch_, stream_));
        } else {
            BCHK(bitnet_hip_gqa_rows_dev(&a, proj, B.main, 1, f32_, pos_, 1, nullptr, 0, stream_));
            BCHK(bitnet_hip_gqa_any_dev(&a, proj, B.main, 1, f32_, pos_, 0, 1, scratch_, stream_));
        }
        BCHK(bitnet_hip_gqa_merge_dev(&a, pos_, 0, 1, scratch_, row, B.ko, 0, stream_));
    } else if (B.mixer) {
        const bitnet_hip_delta d = delta_args(i, pass);
        BCHK(bitnet_hip_delta_step_dev(&d, proj, tail, pos_, row, stream_));
    }
    if (!routed) return gemv(plain_input(row), B.out, B.out_bias, 0, 0, 0, y_[which]);
    const ExpertsSpec &e = S.experts;
    const bitnet_hip_router r = router_args(i);
    float *identity = e.identity ? (float *)(eids_ + 32) : nullptr;
    BCHK(bitnet_hip_experts_up_dev(tail + B.gates, &r, h, B.expert_up.w, e.gated ? 2 * e.ff : e.ff, B.expert_up.cols, B.expert_up.ld,
                                   e.act | (e.gated ? BITNET_HIP_ACT_GATED : 0), eact_, B.expert_down.ld, eids_, identity, stream_));
    BCHK(bitnet_hip_experts_out_dev(B.out.w ? row : nullptr, B.out.w, B.out.cols, B.out.ld, B.out_bias, eact_, B.expert_down.ld, B.expert_down.w, B.expert_down.cols,
                                    B.expert_down.ld, eids_, e.top, width_, identity, h, B.shared ? tail : nullptr, y_[which], stream_));
    return 0;
}

int StackModel::step_latent(size_t i, int pass) {
    const Layer &L = layers_[i];
    const LatentSpec &m = spec_.layers[i].latent;
    TRY(gemv(block_input(L.norm1), L.down_q, nullptr, 0, 0, 0, z_));
    bitnet_hip_vector_input in = plain_input(z_);
    in.kind = BITNET_HIP_IN_NORM, in.eps = spec_.eps, in.weight = L.dq_norm, in.n = m.q_rank;
    bitnet_hip_latent_rows r;
    latent_args(i, pass, z_, L.down_q.rows, nullptr, 0, r);
    TRY(gemv(in, L.uq, nullptr, 0, 0, 0, q_, m.kv_from < 0 ? &r : nullptr));
    TRY(step_attend_latent(i, pass, q_, nullptr, att_, (size_t)m.heads * L.vdimp));
    return gemv(plain_input(att_), L.o, nullptr, 0, 0, 0, y_[0]);
}

// one query q over the latent cache; rows: the position's latent row, still to be written
int StackModel::step_attend_latent(size_t i, int pass, const float *q, const bitnet_hip_latent_rows *rows, float *out, size_t ldo) {
    const Layer &L = layers_[i];
    const bitnet_hip_vector_input qi = plain_input(q);
    BCHK(bitnet_hip_dense_gemv_dev(&qi, L.uk_t.w, L.ldc, L.dimp, L.uk_t.ld, nullptr, 0, 0, 0, qabs_, spec_.layers[i].latent.heads, (size_t)L.ldc * L.uk_t.ld, L.dimp + L.rotp,
                                   L.ldc, rows, f32_, nullptr, stream_));
    bitnet_hip_latent_attention a;
    attention_args(i, pass, a);
    BCHK(bitnet_hip_latent_decode_dev(&a, q, qabs_, pos_, 0, 1, f32_, scratch_, stream_));
    BCHK(bitnet_hip_latent_merge_dev(&a, L.uv.w, pos_, 0, 1, scratch_, out, ldo, 0, stream_));
    return 0;
}

// what the token brings along: norm(W_proj (gelu(W_gate x) * its part of the table's row)) is left to be added
int StackModel::step_side(size_t i) {
    const Layer &L = layers_[i];
    bitnet_hip_epilogue more = {};
    more.mul = side_.w + i * (size_t)spec_.side_dim, more.ld_mul = side_.ld, more.mul_rows = vocab_, more.mul_tokens = history_, more.mul_at = pos_;
    TRY(gemv(block_input(Norm()), L.side_gate, nullptr, BITNET_HIP_ACT_GELU_TANH, 0, 0, act_, nullptr, &more));
    TRY(gemv(plain_input(act_), L.side_proj, nullptr, 0, 0, 0, y_[0]));
    pending_ = Pending();
    pending_.y = y_[0], pending_.w = L.side_norm;
    return 0;
}

int StackModel::step_linear(size_t i, int pass) {
    const Layer &L = layers_[i];
    const LinearSpec &m = spec_.layers[i].linear;
    const size_t split = (size_t)m.heads * (2 * L.dimp + L.vdimp);
    TRY(gemv(block_input(L.norm1), L.qkvg, nullptr, m.act_qkv, m.act_gate, split, lin_));
    BCHK(bitnet_hip_linear_recurrent_dev(lin_, L.qkvg.rows, 1, m.heads, L.dimp, L.vdimp, L.decay_pow, L.slots[(size_t)pass].state, lino_, (size_t)m.heads * L.vdimp, stream_));
    bitnet_hip_vector_input in = plain_input(lino_);
    in.kind = BITNET_HIP_IN_NORM, in.eps = spec_.eps, in.weight = L.out_norm, in.gate = lin_ + split, in.n = m.heads * L.vdimp, in.mean_n = m.heads * m.vdim;
    return gemv(in, L.o, nullptr, 0, 0, 0, y_[0]);
}

// the embedding output of the n tokens from the position on
int StackModel::embed_rows(size_t n, float *out) {
    if (pairs_.w)
        BCHK(bitnet_hip_embed_pairs_bf16_dev(embed_.w, embed_.ld, pairs_.w, pairs_.ld, spec_.pairs.buckets, spec_.pairs.mul_prev, spec_.pairs.mul_cur, history_, pos_, n, width_,
                                             vocab_, spec_.embed_scale, out, stream_));
    else if (embed_norm_)
        BCHK(bitnet_hip_embed_norm_bf16_dev(embed_.w, embed_.ld, history_, pos_, n, width_, vocab_, spec_.embed_scale, embed_norm_, spec_.eps, out, stream_));
    else
        BCHK(bitnet_hip_embed_bf16_dev(embed_.w, embed_.ld, history_, pos_, n, width_, vocab_, spec_.embed_scale, out, stream_));
    return 0;
}

int StackModel::step(bool with_logits, int) {
    cur_ = x0_;
    row_at_ = 0;
    pending_ = Pending();
    TRY(embed_rows(1, x0_));
    for (const Run &run : runs_) {
        const size_t i = run.layer;
        const Layer &L = layers_[i];
        const LayerSpec &S = spec_.layers[i];
        if (run.enters) TRY(step_loop_in());
        TRY(L.block[0].used ? step_block(i, run.pass, 0) : S.mixer == LayerSpec::Latent ? step_latent(i, run.pass) : step_linear(i, run.pass));
        auto leave = [&](int which, const float *norm, const float *scale) {
            const Block &B = L.block[which];
            pending_ = Pending();
            pending_.y = y_[which], pending_.w = norm, pending_.scale = scale;
            if (B.rg) pending_.gate = row_[row_at_] + B.ko + B.fs;
        };
        leave(0, L.norm1b, L.ls1);
        if (!S.parallel && (S.ff > 0 || S.experts.count > 0)) {
            if (L.block[1].used) {
                TRY(step_block(i, run.pass, 1));
            } else {
                bitnet_hip_epilogue more = {};
                more.act_a = L.act_a, more.act_b = L.act_b;
                TRY(gemv(block_input(L.norm2), L.up, L.up_b, S.act_ff | (S.gated ? BITNET_HIP_ACT_GATED : 0), 0, 0, act_, nullptr, &more));
                TRY(gemv(plain_input(act_), L.down, L.down_b, 0, 0, 0, y_[1]));
            }
            leave(1, L.norm2b, L.ls2);
        }
        if (spec_.side_dim > 0) TRY(step_side(i));
    }
    if (with_logits) {
        const bitnet_hip_vector_input in = block_input(final_norm_);
        BCHK(bitnet_hip_dense_logits_dev(&in, head_m_.w, vocab_, head_m_.cols, head_m_.ld, logits_, argmax_, token_, pos_, history_, n_forced_, stream_));
        hidden_ = cur_;
    } else {
        BCHK(bitnet_hip_advance_pos_dev(pos_, stream_));
        hidden_ = nullptr;  // the last sublayer's output was not added: nobody asked for it
    }
    return 0;
}

// ---- a portion of n tokens --------------------------------------------------------------------------------------------

int StackModel::portion_buffers(size_t n) {
    if (n <= rows_cap_) return 0;
    n = up_to(n, 64);
    const size_t es = f32_ ? 4 : 2;
    size_t z = 0, cq = 0, q = 0, qabs = 0, att = 0, act = 0, k = 0, vt = 0, lin = 0, linf = 0, lino = 0, gate = 0, ws = 0, scratch = 0, qf = 0;
    size_t row = 0, tail = 0, qk = 0, v = 0, gates = 0, plan = 0, eact = 0, eout = 0, qc = 0;
    for (size_t i = 0; i < layers_.size(); ++i) {
        const Layer &L = layers_[i];
        const LayerSpec &S = spec_.layers[i];
        if (S.mixer == LayerSpec::Latent) {
            const LatentSpec &m = S.latent;
            const bool direct = m.q_rank == 0;  // (queries in the block's rows)
            if (!direct) {
                z = std::max(z, (size_t)L.down_q.rows);
                cq = std::max(cq, up_to(m.q_rank, 64));
                att = std::max(att, (size_t)L.o.ld);
            }
            if (!f32_ && bitnet_hip_latent_prefill_supported(L.dimp + L.rotp, L.vdimp)) {
                if (!direct) q = std::max(q, (size_t)L.uq.rows);
                k = std::max(k, (size_t)L.uk.rows);
                vt = std::max(vt, (size_t)L.uv.rows);
            } else {
                if (!direct || !f32_) qf = std::max(qf, (size_t)m.heads * (L.dimp + L.rotp));
                qabs = std::max(qabs, (size_t)m.heads * L.ldc);
                scratch = std::max(scratch, bitnet_hip_latent_scratch_bytes(m.heads, L.ldc, kDecodeSlice));
            }
        } else if (S.mixer == LayerSpec::Attention) {
            const AttentionSpec &m = S.attention;
            if (m.taps > 0) qc = std::max(qc, (size_t)m.heads * m.maps * L.dimp);
            if (f32_ || !bitnet_hip_gqa_supported(L.dimp, L.vdimp)) scratch = std::max(scratch, bitnet_hip_gqa_scratch_bytes(m.heads, m.maps, L.vdimp, kDecodeSlice));
        } else if (S.mixer == LayerSpec::Delta) {
            const DeltaSpec &m = S.delta;
            qk = std::max(qk, (size_t)2 * m.kv_heads * L.dimp);
            v = std::max(v, (size_t)m.heads * L.vdimp);
            gates = std::max(gates, (size_t)2 * m.heads);
            if (!f32_ && bitnet_hip_delta_chunked_supported(L.dimp, L.vdimp)) ws = std::max(ws, bitnet_hip_delta_workspace_bytes(n, m.heads, L.dimp, L.vdimp));
        } else {
            const LinearSpec &m = S.linear;
            lino = std::max(lino, (size_t)m.heads * L.vdimp);
            gate = std::max(gate, (size_t)L.o.ld);
            if (!f32_ && bitnet_hip_linear_chunked_supported(L.dimp, L.vdimp)) {
                lin = std::max(lin, (size_t)L.qkvg.rows);
                ws = std::max(ws, bitnet_hip_linear_workspace_bytes(n, m.heads, L.dimp, L.vdimp));
            } else {
                linf = std::max(linf, (size_t)L.qkvg.rows);
            }
        }
        for (const Block &B : L.block) {
            if (!B.used) continue;
            row = std::max(row, up_to((size_t)B.ko + B.fs + B.rg + B.main, 64));
            tail = std::max(tail, up_to(B.tail, 64));
            if (!B.expert_up.w) continue;
            const ExpertsSpec &e = S.experts;
            plan = std::max(plan, bitnet_hip_experts_plan_bytes(n, e.count, e.top));
            eact = std::max(eact, (size_t)e.top * B.expert_down.ld);
            eout = std::max(eout, (size_t)e.top * up_to(width_, 64));
        }
        act = std::max(act, (size_t)std::max(L.down.ld, L.side_proj.ld));
    }
    rows_cap_ = 0;
    if (spec_.loop.times > 0) {
        TRY(grow(px0_, n * width_ * 4));
        TRY(grow(pcat_, n * loop_in_.ld * es));
    }
    TRY(grow(prow_, n * row * es + 256));  // (the latent-space product of f32 rows reads up to 32 columns past a head)
    TRY(grow(pqc_, n * qc * es));
    TRY(grow(ptail_, n * tail * 4));
    TRY(grow(pqk_, n * qk * 4));
    TRY(grow(pv_, n * v * es));
    TRY(grow(pgates_, n * gates * 4));
    TRY(grow(pplan_, plan));
    TRY(grow(peact_, n * eact * es));
    TRY(grow(peout_, n * eout * es));
    TRY(grow(px_, n * width_ * 4));
    TRY(grow(ph_, n * up_to(width_, 64) * es));
    TRY(grow(py_, n * width_ * 4));
    TRY(grow(pz_, n * z * 4));
    TRY(grow(pcq_, n * cq * es));
    TRY(grow(pq_, n * q * 2));
    TRY(grow(pqf_, (n * qf + 64) * 4));  // (the latent-space product reads up to 32 columns past a head)
    TRY(grow(pqabs_, n * qabs * 4));
    TRY(grow(pscratch_, scratch));
    TRY(grow(patt_, n * att * es));
    TRY(grow(pact_, n * act * es));
    TRY(grow(pk_, cap_ * k * 2));
    TRY(grow(pvt_, cap_ * vt * 2));
    TRY(grow(plin_, n * lin * 2));
    TRY(grow(plinf_, n * linf * 4));
    TRY(grow(plino_, n * lino * 4));
    TRY(grow(pgate_, n * gate * es));
    TRY(grow(plws_, ws));
    rows_cap_ = n;
    return 0;
}

int StackModel::matmul(const void *a, size_t lda, bool a_f32, const Matrix &m, const float *bias, size_t n, int act0, int act1, size_t split, void *c,
                       size_t ldc, bool c_f32, const bitnet_hip_epilogue *more) {
    BCHK(bitnet_hip_dense_matmul_dev(a, lda, a_f32, m.w, m.ld, bias, n, m.rows, m.ld, act0, act1, split, c, ldc, c_f32, 1, 0, 0, 0, more, stream_));
    return 0;
}

// rows first .. first + rows - 1 of a block's first product, from ph_
int StackModel::block_matmul(const Layer &L, const Block &B, int first, int rows, size_t n, int act0, int act1, int split, void *c, size_t ldc, bool c_f32) {
    bitnet_hip_epilogue more = {};
    more.act_a = L.act_a, more.act_b = L.act_b;
    BCHK(bitnet_hip_dense_matmul_dev(ph_.p, up_to(width_, 64), f32_, B.in.w + (size_t)first * B.in.ld, B.in.ld, B.in_bias ? B.in_bias + first : nullptr, n, rows, B.in.ld, act0,
                                     act1, split, c, ldc, c_f32, 1, 0, 0, 0, &more, stream_));
    return 0;
}

// The pending sublayer is added to the n rows of px_; h (nullable) receives their norm, or -- x2 given -- [x; x2].
int StackModel::portion_norm(size_t n, const Norm *norm, const float *x2, void *h, size_t ldh) {
    const Pending p = pending_;
    pending_ = Pending();
    // the norm behind the sublayer, and the next one with it where it is of the same kind
    if (p.w && !p.experts && !p.gate && !spec_.center && !x2 && !(h && !norm)) {
        BCHK(bitnet_hip_residual_norm_rows_dev((float *)px_.p, p.y, width_, p.w, p.scale, h ? norm->w : nullptr, spec_.norm_offset, spec_.eps, n, width_, h, ldh, f32_, stream_));
        return 0;
    }
    bitnet_hip_sum_rows r;
    memset(&r, 0, sizeof(r));
    r.x = (float *)px_.p, r.m = n, r.width = width_, r.mult = spec_.residual_mult, r.eps = spec_.eps, r.weight_offset = spec_.norm_offset;
    r.center = spec_.center, r.h_f32 = f32_, r.h = h, r.ldh = ldh, r.x2 = x2;
    if (norm) r.weight = norm->w, r.bias = norm->bias;
    r.y = p.y, r.ldy = width_, r.post_weight = p.w, r.scale = p.scale, r.identity = p.identity, r.input = p.input, r.ld_input = p.input ? up_to(width_, 64) : 0;
    r.y_scale = p.y_scale, r.ld_y_scale = p.ld_y_scale, r.gate = p.gate, r.ld_gate = p.ld_gate;
    if (p.experts) r.expert_rows = peout_.p, r.ld_expert = up_to(width_, 64), r.top = plan_.top, r.slots = plan_.slots, r.slot_weights = plan_.weights;
    BCHK(bitnet_hip_sum_norm_rows_dev(&r, stream_));
    return 0;
}

int StackModel::portion_loop_in(size_t n) {
    TRY(portion_norm(n, nullptr, (const float *)px0_.p, pcat_.p, loop_in_.ld));
    return matmul(pcat_.p, loop_in_.ld, f32_, loop_in_, nullptr, n, 0, 0, 0, px_.p, width_, true);
}

// the sublayers of a block: py_ holds the sum of those that every token takes, the routed experts' rows lie in peout_ by slot
int StackModel::portion_block(size_t i, int pass, int which, size_t n, size_t pos0) {
    const Layer &L = layers_[i];
    const Block &B = L.block[which];
    const LayerSpec &S = spec_.layers[i];
    const size_t ldh = up_to(width_, 64), ld = up_to((size_t)B.ko + B.fs + B.rg + B.main, 64), ldt = up_to(B.tail, 64), es = f32_ ? 4 : 2;
    const bool routed = B.expert_up.w != nullptr;
    char *row = (char *)prow_.p, *gates = row + (size_t)(B.ko + B.fs) * es, *proj = gates + (size_t)B.rg * es;
    float *tail = (float *)ptail_.p;
    const bool prefill_latent = !f32_ && bitnet_hip_latent_prefill_supported(L.dimp + L.rotp, L.vdimp);
    const bool latent = B.mixer && S.mixer == LayerSpec::Latent;
    const int main = latent && !f32_ && !prefill_latent ? 0 : B.main, sig = B.rg ? BITNET_HIP_ACT_SIGMOID : 0;
    if (B.gated) {
        TRY(block_matmul(L, B, 0, B.ff_rows(), n, S.act_ff | BITNET_HIP_ACT_GATED, 0, 0, row + (size_t)B.ko * es, ld, f32_));
        if (B.rg + main > 0) TRY(block_matmul(L, B, B.ff_rows(), B.rg + main, n, sig, 0, B.rg, gates, ld, f32_));
    } else if (B.fs && B.rg && main) {
        TRY(block_matmul(L, B, 0, B.fs + B.rg, n, S.act_ff, sig, B.fs, row + (size_t)B.ko * es, ld, f32_));
        TRY(block_matmul(L, B, B.fs + B.rg, main, n, 0, 0, 0, proj, ld, f32_));
    } else if (B.fs + B.rg + main > 0) {
        TRY(block_matmul(L, B, 0, B.fs + B.rg + main, n, B.fs ? S.act_ff : sig, B.fs ? sig : 0, B.fs ? B.fs : B.rg, row + (size_t)B.ko * es, ld, f32_));
    }
    if (B.tail > 0) TRY(block_matmul(L, B, B.ff_rows() + B.rg + B.main, B.tail, n, B.shared ? BITNET_HIP_ACT_SIGMOID : 0, 0, B.shared, tail, ldt, true));
    if (latent) {
        bitnet_hip_latent_rows r;
        latent_args(i, pass, tail, ldt, nullptr, 0, r);
        if (S.latent.kv_from < 0) BCHK(bitnet_hip_latent_rows_dev(&r, n, f32_, stream_));
        const float *qf = f32_ ? (const float *)proj : (const float *)pqf_.p;
        if (main == 0) TRY(block_matmul(L, B, B.ff_rows() + B.rg, B.main, n, 0, 0, 0, pqf_.p, B.main, true));
        TRY(portion_attend_latent(i, pass, n, pos0, (const uint16_t *)proj, qf, main ? ld : (size_t)B.main, row, ld));
    } else if (B.mixer && S.mixer == LayerSpec::Attention) {
        bitnet_hip_gqa a = gqa_args(i, pass, proj, ld, f32_);
        const bool conv = S.attention.taps > 0;
        const size_t ldq = conv ? a.heads * a.maps * a.dimp : ld;
        const char *q = conv ? (const char *)pqc_.p : proj;
        if (conv) a.taps = S.attention.taps, a.conv = L.conv, a.ring = L.slots[(size_t)pass].ring;
        BCHK(bitnet_hip_gqa_rows_dev(&a, proj, ld, f32_, f32_, pos_, n, conv ? pqc_.p : nullptr, ldq, stream_));
        if (conv) BCHK(bitnet_hip_conv_keep_dev(proj, ld, f32_, L.channels, a.taps, L.slots[(size_t)pass].ring, pos_, n, stream_));
        if (!f32_ && bitnet_hip_gqa_supported(a.dimp, a.vdimp)) {
            BCHK(bitnet_hip_gqa_prefill_dev(&a, (const uint16_t *)q, ldq, pos0 + n, n, (uint16_t *)row, ld, stream_));
        } else {
            for (size_t s = 0; s < n; s += kDecodeSlice) {
                const size_t k = std::min(kDecodeSlice, n - s);
                BCHK(bitnet_hip_gqa_any_dev(&a, q + s * ldq * es, ldq, f32_, f32_, pos_, s, k, (float *)pscratch_.p, stream_));
                BCHK(bitnet_hip_gqa_merge_dev(&a, pos_, s, k, (const float *)pscratch_.p, row + s * ld * es, ld, !f32_, stream_));
                if (a.gate) a.gate = (const char *)a.gate + kDecodeSlice * ld * es;
            }
        }
    } else if (B.mixer) {
        const bitnet_hip_delta d = delta_args(i, pass);
        float *qk = (float *)pqk_.p, *decays = (float *)pgates_.p;
        BCHK(bitnet_hip_delta_rows_dev(&d, proj, ld, f32_, tail, ldt, pos_, n, qk, pv_.p, decays, stream_));
        BCHK(bitnet_hip_delta_keep_dev(&d, proj, ld, f32_, pos_, n, stream_));
        if (!f32_ && bitnet_hip_delta_chunked_supported(L.dimp, L.vdimp))
            BCHK(bitnet_hip_delta_chunked_dev(&d, qk, (const uint16_t *)pv_.p, decays, (const uint16_t *)proj, ld, n, (uint16_t *)row, ld, plws_.p, plws_.bytes, stream_));
        else
            BCHK(bitnet_hip_delta_recurrent_dev(&d, qk, pv_.p, decays, proj, ld, f32_, n, row, ld, stream_));
    }
    if (B.out.w) TRY(matmul(row, ld, f32_, B.out, B.out_bias, n, 0, 0, 0, py_.p, width_, true));
    if (!routed) return 0;
    const ExpertsSpec &e = S.experts;
    const bitnet_hip_router r = router_args(i);
    const size_t tile = !f32_ && n * e.top >= (size_t)96 * e.count ? 128 : 64;
    BCHK(bitnet_hip_experts_plan_make(pplan_.p, pplan_.bytes, n, e.count, e.top, tile, &plan_));
    BCHK(bitnet_hip_experts_route_dev(tail + B.gates, ldt, &r, &plan_, stream_));
    BCHK(bitnet_hip_experts_matmul_dev(&plan_, 1, ph_.p, ldh, f32_, B.expert_up.w, e.gated ? 2 * e.ff : e.ff, B.expert_up.ld, B.expert_up.ld,
                                       e.act | (e.gated ? BITNET_HIP_ACT_GATED : 0), peact_.p, B.expert_down.ld, f32_, stream_));
    BCHK(bitnet_hip_experts_matmul_dev(&plan_, 0, peact_.p, B.expert_down.ld, f32_, B.expert_down.w, width_, B.expert_down.ld, B.expert_down.ld, 0, peout_.p, up_to(width_, 64),
                                       f32_, stream_));
    return 0;
}

int StackModel::portion_latent(size_t i, int pass, size_t n, size_t pos0) {
    const Layer &L = layers_[i];
    const LatentSpec &m = spec_.layers[i].latent;
    const size_t ldh = up_to(width_, 64), ldcq = up_to(m.q_rank, 64), lda = L.o.ld;
    TRY(matmul(ph_.p, ldh, f32_, L.down_q, nullptr, n, 0, 0, 0, pz_.p, L.down_q.rows, true));
    bitnet_hip_latent_rows r;
    latent_args(i, pass, (const float *)pz_.p, L.down_q.rows, pcq_.p, ldcq, r);
    BCHK(bitnet_hip_latent_rows_dev(&r, n, f32_, stream_));
    const bool prefill = !f32_ && bitnet_hip_latent_prefill_supported(L.dimp + L.rotp, L.vdimp);
    TRY(matmul(pcq_.p, ldcq, f32_, L.uq, nullptr, n, 0, 0, 0, prefill ? pq_.p : pqf_.p, L.uq.rows, !prefill));
    TRY(portion_attend_latent(i, pass, n, pos0, (const uint16_t *)pq_.p, (const float *)pqf_.p, L.uq.rows, patt_.p, lda));
    return matmul(patt_.p, lda, f32_, L.o, nullptr, n, 0, 0, 0, py_.p, width_, true);
}

// n queries over the latent cache: q (bf16) where the prompt form covers the heads, qf (f32) elsewhere, both ldq apart
int StackModel::portion_attend_latent(size_t i, int pass, size_t n, size_t pos0, const uint16_t *q, const float *qf, size_t ldq, void *out, size_t ldo) {
    const Layer &L = layers_[i];
    const Slot &K = kv_slot(i, pass);
    const LatentSpec &m = spec_.layers[i].latent;
    const size_t qd = L.dimp + L.rotp, ctx = pos0 + n;
    bitnet_hip_latent_attention a;
    attention_args(i, pass, a);
    a.ldq = ldq;
    if (!f32_ && bitnet_hip_latent_prefill_supported(qd, L.vdimp)) {
        TRY(matmul(K.c, L.ldc, false, L.uk, nullptr, ctx, 0, 0, 0, pk_.p, L.uk.rows, false));
        // the values transposed: W_uv's rows are the product's rows, the cache its "weights"
        BCHK(bitnet_hip_dense_matmul_dev(L.uv.w, L.uv.ld, 0, (const uint16_t *)K.c, L.ldc, nullptr, L.uv.rows, up_to(ctx, 64), L.ldc, 0, 0, 0, pvt_.p, cap_, 0,
                                         1, 0, 0, 0, nullptr, stream_));
        BCHK(bitnet_hip_latent_prefill_dev(&a, q, (const uint16_t *)pk_.p, (const uint16_t *)pvt_.p, cap_, ctx, n, (uint16_t *)out, ldo, stream_));
        return 0;
    }
    // in latent space, a slice of queries at a time
    const size_t es = f32_ ? 4 : 2, ldqa = (size_t)m.heads * L.ldc;
    BCHK(bitnet_hip_dense_matmul_dev(qf, ldq, 1, L.uk_t.w, L.uk_t.ld, nullptr, n, L.ldc, L.uk_t.ld, 0, 0, 0, pqabs_.p, ldqa, 1, m.heads, qd, (size_t)L.ldc * L.uk_t.ld, L.ldc,
                                     nullptr, stream_));
    for (size_t s = 0; s < n; s += kDecodeSlice) {
        const size_t k = std::min(kDecodeSlice, n - s);
        BCHK(bitnet_hip_latent_decode_dev(&a, qf + s * ldq, (const float *)pqabs_.p + s * ldqa, pos_, s, k, f32_, (float *)pscratch_.p, stream_));
        BCHK(bitnet_hip_latent_merge_dev(&a, L.uv.w, pos_, s, k, (const float *)pscratch_.p, (char *)out + s * ldo * es, ldo, !f32_, stream_));
    }
    return 0;
}

int StackModel::portion_side(size_t i, size_t n) {
    const Layer &L = layers_[i];
    TRY(portion_norm(n, nullptr, nullptr, ph_.p, up_to(width_, 64)));
    bitnet_hip_epilogue more = {};
    more.mul = side_.w + i * (size_t)spec_.side_dim, more.ld_mul = side_.ld, more.mul_rows = vocab_, more.mul_tokens = history_, more.mul_at = pos_;
    TRY(matmul(ph_.p, up_to(width_, 64), f32_, L.side_gate, nullptr, n, BITNET_HIP_ACT_GELU_TANH, 0, 0, pact_.p, L.side_proj.ld, f32_, &more));
    TRY(matmul(pact_.p, L.side_proj.ld, f32_, L.side_proj, nullptr, n, 0, 0, 0, py_.p, width_, true));
    pending_ = Pending();
    pending_.y = (const float *)py_.p, pending_.w = L.side_norm;
    return 0;
}

int StackModel::portion_linear(size_t i, int pass, size_t n) {
    const Layer &L = layers_[i];
    float *state = L.slots[(size_t)pass].state;
    const LinearSpec &m = spec_.layers[i].linear;
    const size_t ldh = up_to(width_, 64), ld = L.qkvg.rows, no = (size_t)m.heads * L.vdimp, split = (size_t)m.heads * (2 * L.dimp + L.vdimp);
    const bool chunked = !f32_ && bitnet_hip_linear_chunked_supported(L.dimp, L.vdimp);
    void *lin = chunked ? plin_.p : plinf_.p;
    TRY(matmul(ph_.p, ldh, f32_, L.qkvg, nullptr, n, m.act_qkv, m.act_gate, split, lin, ld, !chunked));
    const void *gate = chunked ? (const void *)((const uint16_t *)lin + split) : (const void *)((const float *)lin + split);
    if (chunked)
        BCHK(bitnet_hip_linear_chunked_dev((const uint16_t *)lin, ld, n, m.heads, L.dimp, L.vdimp, L.decay_pow, state, (float *)plino_.p, no, plws_.p, plws_.bytes,
                                           stream_));
    else
        BCHK(bitnet_hip_linear_recurrent_dev((const float *)lin, ld, n, m.heads, L.dimp, L.vdimp, L.decay_pow, state, (float *)plino_.p, no, stream_));
    BCHK(bitnet_hip_gated_norm_rows_dev((const float *)plino_.p, no, L.out_norm, gate, ld, spec_.eps, !chunked, n, no, (size_t)m.heads * m.vdim, pgate_.p, L.o.ld,
                                        f32_, stream_));
    return matmul(pgate_.p, L.o.ld, f32_, L.o, nullptr, n, 0, 0, 0, py_.p, width_, true);
}

// tokens pos0 .. pos0 + n - 1 of the history through every layer; px_ holds the residual stream, *pos_ stays at pos0
int StackModel::portion(int rows, int pos0) {
    const size_t n = rows, ldh = up_to(width_, 64);
    TRY(portion_buffers(n));
    float *x = (float *)px_.p;
    const float *y = (const float *)py_.p;
    TRY(embed_rows(n, x));
    if (spec_.loop.times > 0) TRY(embed_rows(n, (float *)px0_.p));
    pending_ = Pending();
    for (const Run &run : runs_) {
        const size_t i = run.layer;
        const Layer &L = layers_[i];
        const LayerSpec &S = spec_.layers[i];
        if (run.enters) TRY(portion_loop_in(n));
        TRY(portion_norm(n, &L.norm1, nullptr, ph_.p, ldh));
        TRY(L.block[0].used ? portion_block(i, run.pass, 0, n, pos0) : S.mixer == LayerSpec::Latent ? portion_latent(i, run.pass, n, pos0) : portion_linear(i, run.pass, n));
        auto leave = [&](int which, const Norm &ahead, const float *norm, const float *scale) {
            const Block &B = L.block[which];
            const bool routed = B.expert_up.w != nullptr;
            Pending p;
            p.y = routed && !B.out.w ? nullptr : y, p.w = norm, p.scale = scale;
            p.experts = routed, p.input = ahead.w ? ph_.p : nullptr, p.identity = S.experts.identity > 0;
            if (B.rg) p.gate = (const char *)prow_.p + (size_t)(B.ko + B.fs) * (f32_ ? 4 : 2), p.ld_gate = up_to((size_t)B.ko + B.fs + B.rg + B.main, 64);
            if (B.shared) p.y_scale = (const float *)ptail_.p, p.ld_y_scale = up_to(B.tail, 64);
            pending_ = p;
        };
        leave(0, L.norm1, L.norm1b, L.ls1);
        if (!S.parallel && (S.ff > 0 || S.experts.count > 0)) {
            TRY(portion_norm(n, &L.norm2, nullptr, ph_.p, ldh));
            if (L.block[1].used) {
                TRY(portion_block(i, run.pass, 1, n, pos0));
            } else {
                bitnet_hip_epilogue more = {};
                more.act_a = L.act_a, more.act_b = L.act_b;
                TRY(matmul(ph_.p, ldh, f32_, L.up, L.up_b, n, S.act_ff | (S.gated ? BITNET_HIP_ACT_GATED : 0), 0, 0, pact_.p, L.down.ld, f32_, &more));
                TRY(matmul(pact_.p, L.down.ld, f32_, L.down, L.down_b, n, 0, 0, 0, py_.p, width_, true));
            }
            leave(1, L.norm2, L.norm2b, L.ls2);
        }
        if (spec_.side_dim > 0) TRY(portion_side(i, n));
    }
    TRY(portion_norm(n, nullptr, nullptr, nullptr, 0));
    hidden_ = x + (n - 1) * (size_t)width_;
    return 0;
}

int StackModel::set_position(int p) {
    HCHK(hipMemcpyAsync(pos_, &p, 4, hipMemcpyHostToDevice, (hipStream_t)stream_));
    HCHK(hipStreamSynchronize((hipStream_t)stream_));  // `p` is a stack variable
    return 0;
}

int StackModel::prefill(int n, bool with_logits, int, float *elapsed_ms) {
    if (!ready()) return fail_arg("model globals not set");
    const int p = position();
    if (p < 0) return BITNET_HIP_ERR_GPU;
    if (n <= 0 || p + n > host_forced_) return fail_arg("prefill: feed() the prompt tokens first");
    if (p + n > max_pos_ - 1) return fail_arg("KV cache overflow");
    TRY(portion_buffers(n));
    hipStream_t s = (hipStream_t)stream_;
    Event e0, e1;
    HCHK(hipEventCreate(&e0.e));
    HCHK(hipEventCreate(&e1.e));
    HCHK(hipEventRecord(e0.e, s));
    TRY(portion(n, p));
    TRY(set_position(with_logits ? p + n - 1 : p + n));
    if (with_logits) {
        bitnet_hip_vector_input in = plain_input(hidden_);
        in.kind = BITNET_HIP_IN_NORM;
        in.eps = spec_.eps, in.weight_offset = spec_.norm_offset, in.weight = final_norm_.w, in.bias = final_norm_.bias, in.center = spec_.center, in.n = width_;
        BCHK(bitnet_hip_dense_logits_dev(&in, head_m_.w, vocab_, head_m_.cols, head_m_.ld, logits_, argmax_, token_, pos_, history_, n_forced_, s));
    }
    HCHK(hipEventRecord(e1.e, s));
    HCHK(hipStreamSynchronize(s));
    float ms = 0.f;
    HCHK(hipEventElapsedTime(&ms, e0.e, e1.e));
    if (elapsed_ms) *elapsed_ms = ms;
    return 0;
}

int StackModel::forward(const int32_t *tokens, int n, const int32_t *want, int n_want, float *logits) {
    if (n <= 1) return Sequence::forward(tokens, n, want, n_want, logits);
    if (n_want < 0 || (n_want > 0 && (!want || !logits))) return fail_arg("forward: null pointer");
    for (int w = 0; w < n_want; ++w)
        if (want[w] < 0 || want[w] >= n) return fail_arg("forward: a wanted place is not among the tokens");
    TRY(feed(tokens, n));
    TRY(prefill(n, false, 0, nullptr));
    if (n_want == 0) return 0;
    const size_t k = n_want, ldh = up_to(width_, 64), es = f32_ ? 4 : 2;
    TRY(grow(pwant_, k * 4));
    TRY(grow(pxw_, k * width_ * 4));
    TRY(grow(phw_, k * ldh * es));
    TRY(grow(plog_, k * vocab_ * 4));
    hipStream_t s = (hipStream_t)stream_;
    HCHK(hipMemcpy(pwant_.p, want, k * 4, hipMemcpyHostToDevice));
    BCHK(bitnet_hip_gather_rows_dev((const float *)px_.p, (const int32_t *)pwant_.p, k, width_, (float *)pxw_.p, s));
    bitnet_hip_sum_rows r;
    memset(&r, 0, sizeof(r));
    r.x = (float *)pxw_.p, r.m = k, r.width = width_, r.eps = spec_.eps, r.weight_offset = spec_.norm_offset, r.center = spec_.center, r.h_f32 = f32_;
    r.weight = final_norm_.w, r.bias = final_norm_.bias, r.h = phw_.p, r.ldh = ldh;
    BCHK(bitnet_hip_sum_norm_rows_dev(&r, s));
    TRY(matmul(phw_.p, ldh, f32_, head_m_, nullptr, k, 0, 0, 0, plog_.p, vocab_, true));
    HCHK(hipStreamSynchronize(s));
    HCHK(hipMemcpy(logits, plog_.p, k * vocab_ * 4, hipMemcpyDeviceToHost));
    return 0;
}

int StackModel::last_hidden(float *out) {
    if (!hidden_ || !out) return fail_arg("last_hidden: the last step ran without logits");
    HCHK(hipMemcpy(out, hidden_, (size_t)width_ * 4, hipMemcpyDeviceToHost));
    return 0;
}

}  // namespace bitnet_host
