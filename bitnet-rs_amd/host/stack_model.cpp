// stack_model.cpp -- see stack_model.hpp.  Host orchestration only: every device operation is a bitnet_hip_* call or plain HIP
// memory plumbing.
#include "stack_model.hpp"

#include <algorithm>
#include <cmath>
#include <cstdio>
#include <cstring>

namespace bitnet_host {

namespace {
constexpr size_t kDecodeSlice = 64;  // queries per latent-space attention call of a portion
size_t up_to(size_t v, size_t a) { return (v + a - 1) / a * a; }
}  // namespace

std::vector<double> rotary_frequencies(const RotarySpec &r, double *mult) {
    std::vector<double> f((size_t)r.dims / 2);
    for (size_t i = 0; i < f.size(); ++i) f[i] = std::pow(r.base, -2.0 * (double)i / r.dims);
    *mult = 1.0;
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
    if (init_sequence(spec.vocab, spec.width, max_pos) != 0) return;
    cap_ = up_to((size_t)max_pos + 1, 64);
    size_t z = 64, q = 64, qabs = 64, att = 64, act = 64, lin = 64, lino = 64, scratch = 64;
    const size_t es = f32_ ? 4 : 2;
    for (size_t i = 0; i < layers_.size(); ++i) {
        Layer &L = layers_[i];
        const LayerSpec &S = spec_.layers[i];
        if (S.mixer == LayerSpec::Latent) {
            const LatentSpec &m = S.latent;
            if (m.rot_dim != m.rot.dims || m.rot_dim % 2 || m.rot_dim > 256) {
                err_ = "stack: the rotated part must be even, at most 256 and rotated whole";
                return;
            }
            if (m.kv_from >= 0) {
                const LayerSpec *src = (size_t)m.kv_from < i ? &spec_.layers[(size_t)m.kv_from] : nullptr;
                if (!src || src->mixer != LayerSpec::Latent || src->latent.kv_from >= 0 || src->latent.kv_rank != m.kv_rank || !(src->latent.rot == m.rot)) {
                    err_ = "stack: layer " + std::to_string(i) + " reads the cache of layer " + std::to_string(m.kv_from) + ", which has none that fits";
                    return;
                }
            }
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
        } else {
            const LinearSpec &m = S.linear;
            L.dimp = (int)up_to(m.dim, 32), L.vdimp = (int)up_to(m.vdim, 32);
            if (L.dimp > 512 || m.decay.size() != (size_t)m.heads) {
                err_ = "stack: linear attention: head of more than 512 columns, or not one decay per head";
                return;
            }
            lin = std::max(lin, (size_t)m.heads * 2 * (L.dimp + L.vdimp));
            lino = std::max(lino, (size_t)m.heads * L.vdimp);
        }
        act = std::max(act, (size_t)S.ff);
    }
    auto alloc = [&](void **p, size_t bytes) {
        if (hipMalloc(p, bytes) != hipSuccess || hipMemset(*p, 0, bytes) != hipSuccess) return false;
        owned_.push_back(*p);
        return true;
    };
    auto vec = [&](float **p, size_t n) { return alloc((void **)p, up_to(n, 64) * 4); };
    bool ok = vec(&x_[0], width_) && vec(&x_[1], width_) && vec(&y_[0], width_) && vec(&y_[1], width_) && vec(&z_, z) && vec(&q_, q) && vec(&qabs_, qabs) &&
              vec(&att_, att) && vec(&act_, act) && vec(&lin_, lin) && vec(&lino_, lino) && vec(&scratch_, scratch) && alloc(&argmax_, 8192);
    for (size_t i = 0; ok && i < layers_.size(); ++i) {
        Layer &L = layers_[i];
        const LayerSpec &S = spec_.layers[i];
        if (S.mixer == LayerSpec::Latent) {
            if (S.latent.kv_from < 0) ok = alloc(&L.cache.c, cap_ * L.ldc * es) && alloc(&L.cache.r, cap_ * L.rotp * es);
            ok = ok && rope_tables(S.latent.rot, &L.cos, &L.sin) == 0;
        } else {
            ok = alloc((void **)&L.state, (size_t)S.linear.heads * L.dimp * L.vdimp * 4);
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
                      &pwant_, &pxw_, &phw_, &plog_})
        if (b->p) hipFree(b->p);
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
    if (w.norm1.size() != W || w.norm1b.size() != W || (!w.ls1.empty() && w.ls1.size() != W)) return fail_arg("stack: norm of the wrong size");
    TRY(upload(&L.norm1, w.norm1));
    TRY(upload(&L.norm1b, w.norm1b));
    TRY(upload(&L.ls1, w.ls1));
    if (S.mixer == LayerSpec::Latent) {
        const LatentSpec &m = S.latent;
        const size_t H = m.heads, D = m.dim, R = m.rot_dim, V = m.vdim;
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
        // W_uk twice: as it is (the prompt expands keys) and per head transposed (a step takes the query into latent space)
        TRY(upload_matrix(L.uk, pad_rows(w.uk, H, D, L.dimp, m.kv_rank), (int)(H * L.dimp), m.kv_rank));
        t.assign(H * L.ldc * L.dimp, 0);
        for (size_t h = 0; h < H; ++h)
            for (size_t d = 0; d < D; ++d)
                for (size_t c = 0; c < (size_t)m.kv_rank; ++c) t[(h * L.ldc + c) * L.dimp + d] = w.uk[(h * D + d) * m.kv_rank + c];
        TRY(upload_matrix(L.uk_t, t, (int)(H * L.ldc), L.dimp));
        weight_bytes_ -= t.size() * 2;  // one of the two copies is read per token
        TRY(upload_matrix(L.uv, pad_rows(w.uv, H, V, L.vdimp, m.kv_rank), (int)(H * L.vdimp), m.kv_rank));
        TRY(upload_matrix(L.o, pad_cols(w.o, W, H, V, L.vdimp), (int)W, (int)(H * L.vdimp)));
        TRY(upload(&L.dq_norm, w.dq_norm));
        TRY(upload(&L.dkv_norm, w.dkv_norm));
        TRY(upload(&L.sink, w.sink));
    } else {
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
    if (S.ff > 0) {
        const size_t F = S.ff;
        if (w.norm2.size() != W || w.norm2b.size() != W || (!w.ls2.empty() && w.ls2.size() != W) || !w.up || !w.down || (!w.up_b.empty() && w.up_b.size() != F) ||
            (!w.down_b.empty() && w.down_b.size() != W))
            return fail_arg("stack: incomplete feed-forward weights");
        TRY(upload(&L.norm2, w.norm2));
        TRY(upload(&L.norm2b, w.norm2b));
        TRY(upload(&L.ls2, w.ls2));
        TRY(upload_matrix(L.up, take(w.up, F * W), (int)F, (int)W));
        TRY(upload_matrix(L.down, take(w.down, W * F), (int)W, (int)F));
        TRY(upload(&L.up_b, w.up_b));
        TRY(upload(&L.down_b, w.down_b));
    }
    L.set = true;
    ++layers_set_;
    return 0;
}

int StackModel::set_globals(const uint16_t *embed, const std::vector<float> &final_norm, const uint16_t *head) {
    if (!embed || final_norm.size() != (size_t)width_ || !head) return fail_arg("stack: incomplete globals");
    if (head_) return fail_arg("the model already holds its globals");
    const size_t n = (size_t)vocab_ * width_;
    TRY(upload_matrix(embed_, take(embed, n), vocab_, width_));
    weight_bytes_ -= n * 2;  // a row of it is read per token
    TRY(upload_matrix(head_m_, take(head, n), vocab_, width_));
    TRY(upload(&final_norm_, final_norm));
    head_ = head_m_.w;
    return 0;
}

int StackModel::clear_state() {
    // the caches need no clearing: a position is read only after it was written, what lies past it meets a zero weight
    for (size_t i = 0; i < layers_.size(); ++i)
        if (layers_[i].state)
            HCHK(hipMemsetAsync(layers_[i].state, 0, (size_t)spec_.layers[i].linear.heads * layers_[i].dimp * layers_[i].vdimp * 4, (hipStream_t)stream_));
    HCHK(hipStreamSynchronize((hipStream_t)stream_));
    hidden_ = nullptr;
    return 0;
}

void StackModel::attention_args(size_t i, bitnet_hip_latent_attention &a) const {
    const Layer &L = layers_[i], &K = kv_layer(i);
    const LatentSpec &m = spec_.layers[i].latent;
    a.heads = m.heads, a.dimp = L.dimp, a.qd = L.dimp + L.rotp, a.vdimp = L.vdimp, a.kv_rank = m.kv_rank, a.rot_dim = m.rot_dim;
    a.scale = m.scale, a.sink = L.sink, a.ccache = K.cache.c, a.rcache = K.cache.r, a.ldc = L.ldc, a.ldr = L.rotp, a.capacity = cap_;
    a.rope_cos = L.cos, a.rope_sin = L.sin;
}

void StackModel::latent_args(size_t i, const float *z, size_t ldz, void *cq, size_t ldcq, bitnet_hip_latent_rows &r) const {
    const Layer &L = layers_[i];
    const LatentSpec &m = spec_.layers[i].latent;
    memset(&r, 0, sizeof(r));
    r.z = z, r.ldz = ldz, r.q_rank = m.q_rank, r.q_weight = L.dq_norm, r.eps = spec_.eps, r.cq = cq, r.ldcq = ldcq, r.pos = pos_;
    if (m.kv_from < 0) {
        r.kv_rank = m.kv_rank, r.rot_dim = m.rot_dim, r.kv_weight = L.dkv_norm;
        r.ccache = L.cache.c, r.rcache = L.cache.r, r.ldc = L.ldc, r.ldr = L.rotp, r.rope_cos = L.cos, r.rope_sin = L.sin;
    }
}

// ---- one token --------------------------------------------------------------------------------------------------------
// x_[cur_] is the residual stream up to the pending sublayer; the launch that normalises it for the next sublayer adds the pending
// output on the way and leaves the sum in the other buffer.

int StackModel::gemv(const bitnet_hip_vector_input &in, const Matrix &m, const float *bias, int act0, int act1, size_t split, float *y,
                     const bitnet_hip_latent_rows *latent) {
    BCHK(bitnet_hip_dense_gemv_dev(&in, m.w, m.rows, m.cols, m.ld, bias, act0, act1, split, y, 1, 0, 0, 0, latent, f32_, stream_));
    return 0;
}

static bitnet_hip_vector_input plain_input(const float *x) {
    bitnet_hip_vector_input in;
    memset(&in, 0, sizeof(in));
    in.x = x;
    in.kind = BITNET_HIP_IN_PLAIN;
    return in;
}

bitnet_hip_vector_input StackModel::block_input(const float *norm) {
    bitnet_hip_vector_input in = plain_input(x_[cur_]);
    in.kind = BITNET_HIP_IN_RESIDUAL_NORM;
    in.eps = spec_.eps, in.weight_offset = spec_.norm_offset, in.weight = norm, in.n = width_;
    if (pending_.y) {
        cur_ ^= 1;
        in.y = pending_.y, in.post_weight = pending_.w, in.scale = pending_.scale, in.x_out = x_[cur_];
        pending_ = Pending();
    }
    return in;
}

int StackModel::step_latent(size_t i) {
    const Layer &L = layers_[i];
    const LatentSpec &m = spec_.layers[i].latent;
    TRY(gemv(block_input(L.norm1), L.down_q, nullptr, 0, 0, 0, z_));
    bitnet_hip_vector_input in = plain_input(z_);
    in.kind = BITNET_HIP_IN_NORM, in.eps = spec_.eps, in.weight = L.dq_norm, in.n = m.q_rank;
    bitnet_hip_latent_rows r;
    latent_args(i, z_, L.down_q.rows, nullptr, 0, r);
    TRY(gemv(in, L.uq, nullptr, 0, 0, 0, q_, m.kv_from < 0 ? &r : nullptr));
    const size_t qd = L.dimp + L.rotp;
    const bitnet_hip_vector_input qi = plain_input(q_);
    BCHK(bitnet_hip_dense_gemv_dev(&qi, L.uk_t.w, L.ldc, L.dimp, L.uk_t.ld, nullptr, 0, 0, 0, qabs_, m.heads, (size_t)L.ldc * L.uk_t.ld, qd, L.ldc, nullptr, 0,
                                   stream_));
    bitnet_hip_latent_attention a;
    attention_args(i, a);
    BCHK(bitnet_hip_latent_decode_dev(&a, q_, qabs_, pos_, 0, 1, f32_, scratch_, stream_));
    BCHK(bitnet_hip_latent_merge_dev(&a, L.uv.w, pos_, 0, 1, scratch_, att_, (size_t)m.heads * L.vdimp, 0, stream_));
    return gemv(plain_input(att_), L.o, nullptr, 0, 0, 0, y_[0]);
}

int StackModel::step_linear(size_t i) {
    const Layer &L = layers_[i];
    const LinearSpec &m = spec_.layers[i].linear;
    const size_t split = (size_t)m.heads * (2 * L.dimp + L.vdimp);
    TRY(gemv(block_input(L.norm1), L.qkvg, nullptr, m.act_qkv, m.act_gate, split, lin_));
    BCHK(bitnet_hip_linear_recurrent_dev(lin_, L.qkvg.rows, 1, m.heads, L.dimp, L.vdimp, L.decay_pow, L.state, lino_, (size_t)m.heads * L.vdimp, stream_));
    bitnet_hip_vector_input in = plain_input(lino_);
    in.kind = BITNET_HIP_IN_NORM, in.eps = spec_.eps, in.weight = L.out_norm, in.gate = lin_ + split, in.n = m.heads * L.vdimp, in.mean_n = m.heads * m.vdim;
    return gemv(in, L.o, nullptr, 0, 0, 0, y_[0]);
}

int StackModel::step(bool with_logits, int) {
    cur_ = 0;
    pending_ = Pending();
    BCHK(bitnet_hip_embed_bf16_dev(embed_.w, embed_.ld, history_, pos_, 1, width_, vocab_, x_[0], stream_));
    for (size_t i = 0; i < layers_.size(); ++i) {
        const Layer &L = layers_[i];
        const LayerSpec &S = spec_.layers[i];
        TRY(S.mixer == LayerSpec::Latent ? step_latent(i) : step_linear(i));
        pending_ = {y_[0], L.norm1b, L.ls1};
        if (S.ff > 0) {
            TRY(gemv(block_input(L.norm2), L.up, L.up_b, S.act_ff, 0, 0, act_));
            TRY(gemv(plain_input(act_), L.down, L.down_b, 0, 0, 0, y_[1]));
            pending_ = {y_[1], L.norm2b, L.ls2};
        }
    }
    if (with_logits) {
        const bitnet_hip_vector_input in = block_input(final_norm_);
        BCHK(bitnet_hip_dense_logits_dev(&in, head_m_.w, vocab_, head_m_.cols, head_m_.ld, logits_, argmax_, token_, pos_, history_, n_forced_, stream_));
        hidden_ = x_[cur_];
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
    for (size_t i = 0; i < layers_.size(); ++i) {
        const Layer &L = layers_[i];
        const LayerSpec &S = spec_.layers[i];
        if (S.mixer == LayerSpec::Latent) {
            const LatentSpec &m = S.latent;
            z = std::max(z, (size_t)L.down_q.rows);
            cq = std::max(cq, up_to(m.q_rank, 64));
            att = std::max(att, (size_t)L.o.ld);
            if (!f32_ && bitnet_hip_latent_prefill_supported(L.dimp + L.rotp, L.vdimp)) {
                q = std::max(q, (size_t)L.uq.rows);
                k = std::max(k, (size_t)L.uk.rows);
                vt = std::max(vt, (size_t)L.uv.rows);
            } else {
                qf = std::max(qf, (size_t)L.uq.rows);
                qabs = std::max(qabs, (size_t)m.heads * L.ldc);
                scratch = std::max(scratch, bitnet_hip_latent_scratch_bytes(m.heads, L.ldc, kDecodeSlice));
            }
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
        act = std::max(act, S.ff ? (size_t)L.down.ld : 0);
    }
    rows_cap_ = 0;
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
                       size_t ldc, bool c_f32) {
    BCHK(bitnet_hip_dense_matmul_dev(a, lda, a_f32, m.w, m.ld, bias, n, m.rows, m.ld, act0, act1, split, c, ldc, c_f32, 1, 0, 0, 0, stream_));
    return 0;
}

int StackModel::portion_latent(size_t i, size_t n, size_t pos0) {
    const Layer &L = layers_[i], &K = kv_layer(i);
    const LatentSpec &m = spec_.layers[i].latent;
    const size_t ldh = up_to(width_, 64), ldcq = up_to(m.q_rank, 64), qd = L.dimp + L.rotp, lda = L.o.ld, ctx = pos0 + n;
    TRY(matmul(ph_.p, ldh, f32_, L.down_q, nullptr, n, 0, 0, 0, pz_.p, L.down_q.rows, true));
    bitnet_hip_latent_rows r;
    latent_args(i, (const float *)pz_.p, L.down_q.rows, pcq_.p, ldcq, r);
    BCHK(bitnet_hip_latent_rows_dev(&r, n, f32_, stream_));
    bitnet_hip_latent_attention a;
    attention_args(i, a);
    if (!f32_ && bitnet_hip_latent_prefill_supported(qd, L.vdimp)) {
        TRY(matmul(pcq_.p, ldcq, false, L.uq, nullptr, n, 0, 0, 0, pq_.p, L.uq.rows, false));
        TRY(matmul(K.cache.c, L.ldc, false, L.uk, nullptr, ctx, 0, 0, 0, pk_.p, L.uk.rows, false));
        // the values transposed: W_uv's rows are the product's rows, the cache its "weights"
        BCHK(bitnet_hip_dense_matmul_dev(L.uv.w, L.uv.ld, 0, (const uint16_t *)K.cache.c, L.ldc, nullptr, L.uv.rows, up_to(ctx, 64), L.ldc, 0, 0, 0, pvt_.p, cap_, 0,
                                         1, 0, 0, 0, stream_));
        BCHK(bitnet_hip_latent_prefill_dev(&a, (const uint16_t *)pq_.p, (const uint16_t *)pk_.p, (const uint16_t *)pvt_.p, cap_, ctx, n, (uint16_t *)patt_.p, lda,
                                           stream_));
    } else {
        // in latent space, a slice of queries at a time
        const size_t es = f32_ ? 4 : 2, ldq = L.uq.rows, ldqa = (size_t)m.heads * L.ldc;
        TRY(matmul(pcq_.p, ldcq, f32_, L.uq, nullptr, n, 0, 0, 0, pqf_.p, ldq, true));
        BCHK(bitnet_hip_dense_matmul_dev(pqf_.p, ldq, 1, L.uk_t.w, L.uk_t.ld, nullptr, n, L.ldc, L.uk_t.ld, 0, 0, 0, pqabs_.p, ldqa, 1, m.heads, qd,
                                         (size_t)L.ldc * L.uk_t.ld, L.ldc, stream_));
        for (size_t s = 0; s < n; s += kDecodeSlice) {
            const size_t k = std::min(kDecodeSlice, n - s);
            BCHK(bitnet_hip_latent_decode_dev(&a, (const float *)pqf_.p + s * ldq, (const float *)pqabs_.p + s * ldqa, pos_, s, k, f32_, (float *)pscratch_.p, stream_));
            BCHK(bitnet_hip_latent_merge_dev(&a, L.uv.w, pos_, s, k, (const float *)pscratch_.p, (char *)patt_.p + s * lda * es, lda, !f32_, stream_));
        }
    }
    return matmul(patt_.p, lda, f32_, L.o, nullptr, n, 0, 0, 0, py_.p, width_, true);
}

int StackModel::portion_linear(size_t i, size_t n) {
    const Layer &L = layers_[i];
    const LinearSpec &m = spec_.layers[i].linear;
    const size_t ldh = up_to(width_, 64), ld = L.qkvg.rows, no = (size_t)m.heads * L.vdimp, split = (size_t)m.heads * (2 * L.dimp + L.vdimp);
    const bool chunked = !f32_ && bitnet_hip_linear_chunked_supported(L.dimp, L.vdimp);
    void *lin = chunked ? plin_.p : plinf_.p;
    TRY(matmul(ph_.p, ldh, f32_, L.qkvg, nullptr, n, m.act_qkv, m.act_gate, split, lin, ld, !chunked));
    const void *gate = chunked ? (const void *)((const uint16_t *)lin + split) : (const void *)((const float *)lin + split);
    if (chunked)
        BCHK(bitnet_hip_linear_chunked_dev((const uint16_t *)lin, ld, n, m.heads, L.dimp, L.vdimp, L.decay_pow, L.state, (float *)plino_.p, no, plws_.p, plws_.bytes,
                                           stream_));
    else
        BCHK(bitnet_hip_linear_recurrent_dev((const float *)lin, ld, n, m.heads, L.dimp, L.vdimp, L.decay_pow, L.state, (float *)plino_.p, no, stream_));
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
    BCHK(bitnet_hip_embed_bf16_dev(embed_.w, embed_.ld, history_, pos_, n, width_, vocab_, x, stream_));
    const float *post = nullptr, *scale = nullptr;
    bool have = false;
    for (size_t i = 0; i < layers_.size(); ++i) {
        const Layer &L = layers_[i];
        const LayerSpec &S = spec_.layers[i];
        BCHK(bitnet_hip_residual_norm_rows_dev(x, have ? y : nullptr, width_, post, scale, L.norm1, spec_.norm_offset, spec_.eps, n, width_, ph_.p, ldh, f32_, stream_));
        TRY(S.mixer == LayerSpec::Latent ? portion_latent(i, n, pos0) : portion_linear(i, n));
        have = true, post = L.norm1b, scale = L.ls1;
        if (S.ff > 0) {
            BCHK(bitnet_hip_residual_norm_rows_dev(x, y, width_, post, scale, L.norm2, spec_.norm_offset, spec_.eps, n, width_, ph_.p, ldh, f32_, stream_));
            TRY(matmul(ph_.p, ldh, f32_, L.up, L.up_b, n, S.act_ff, 0, 0, pact_.p, L.down.ld, f32_));
            TRY(matmul(pact_.p, L.down.ld, f32_, L.down, L.down_b, n, 0, 0, 0, py_.p, width_, true));
            post = L.norm2b, scale = L.ls2;
        }
    }
    BCHK(bitnet_hip_residual_norm_rows_dev(x, y, width_, post, scale, nullptr, spec_.norm_offset, spec_.eps, n, width_, nullptr, 0, 0, stream_));
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
        in.eps = spec_.eps, in.weight_offset = spec_.norm_offset, in.weight = final_norm_, in.n = width_;
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
    BCHK(bitnet_hip_residual_norm_rows_dev((float *)pxw_.p, nullptr, 0, nullptr, nullptr, final_norm_, spec_.norm_offset, spec_.eps, k, width_, phw_.p, ldh, f32_, s));
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
