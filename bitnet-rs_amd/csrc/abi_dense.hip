// abi_dense.hip -- section 5 of include/bitnet_hip.h, first part: bf16-weight operators, latent and linear attention.  Shapes are checked here against
// what the kernels assume; the kernels live in kernels_dense.hip, kernels_latent.hip and kernels_linear.hip.
#include "dense.hpp"

using namespace bitnet_hip;

static_assert(kLinBlock == BITNET_HIP_LINEAR_BLOCK, "the decay table's length is part of the interface");

#define BH_REQUIRE(cond, ...)                                                      \
    do {                                                                           \
        if (!(cond)) return set_error(BITNET_HIP_ERR_INVALID_ARGUMENT, __VA_ARGS__); \
    } while (0)

namespace {
bool act_ok(int a) { return a >= BITNET_HIP_ACT_NONE && a <= BITNET_HIP_ACT_XIELU; }

int to_latent_rows(const bitnet_hip_latent_rows *r, size_t m, int f32, LatentRows &o) {
    BH_REQUIRE(r && r->z && r->pos, "latent_rows: null pointer");
    BH_REQUIRE(m > 0 && r->q_rank >= 0 && r->kv_rank >= 0, "latent_rows: bad sizes");
    BH_REQUIRE(r->ldz >= (size_t)r->q_rank + (r->kv_rank ? r->kv_rank + r->rot_dim : 0), "latent_rows: ldz %zu too short", r->ldz);
    if (r->cq) BH_REQUIRE(r->q_weight && r->q_rank > 0 && r->ldcq >= (size_t)r->q_rank, "latent_rows: bad query latent");
    if (r->kv_rank)
        BH_REQUIRE(r->kv_weight && r->ccache && r->rcache && r->rope_cos && r->rope_sin && r->ldc >= (size_t)r->kv_rank && r->rot_dim % 2 == 0 &&
                       r->rot_dim >= 0 && r->ldr >= (size_t)r->rot_dim,
                   "latent_rows: bad key latent");
    o.z = r->z, o.ldz = (int)r->ldz, o.q_rank = r->q_rank, o.kv_rank = r->kv_rank, o.rot_dim = r->rot_dim;
    o.q_weight = r->q_weight, o.kv_weight = r->kv_weight, o.eps = r->eps;
    o.cq = r->cq, o.ldcq = (int)r->ldcq, o.ccache = r->ccache, o.rcache = r->rcache, o.ldc = (int)r->ldc, o.ldr = (int)r->ldr;
    o.rope_cos = r->rope_cos, o.rope_sin = r->rope_sin, o.pos = r->pos, o.m = (int)m, o.f32 = f32;
    return 0;
}

// rows: those of W ahead of pairing; m: rows of the output
int to_epilogue(const bitnet_hip_epilogue *e, size_t rows, Epilogue &o) {
    if (!e) return 0;
    BH_REQUIRE(act_ok(e->act2) && e->pairs <= rows && e->pairs % 4 == 0, "product: bad pairs or third activation");
    if (e->taps) {
        BH_REQUIRE(e->conv && e->ring && e->pos && e->channels > 0 && e->taps <= (size_t)kMaxTaps && e->conv_from + e->channels <= rows && e->conv_from >= e->pairs,
                   "product: bad convolution (%zu taps, rows %zu + %zu of %zu)", e->taps, e->conv_from, e->channels, rows);
        o.conv_from = (int)e->conv_from, o.channels = (int)e->channels, o.taps = (int)e->taps, o.conv = e->conv, o.ring = e->ring, o.pos = e->pos;
    }
    if (e->mul) {
        BH_REQUIRE(e->pairs == 0 && e->mul_tokens && e->mul_at && e->mul_rows > 0 && e->ld_mul >= rows, "product: bad table of factors");
        BH_CHECK_DIMS(e->mul_rows, e->ld_mul);
        o.mul = e->mul, o.ld_mul = e->ld_mul, o.mul_rows = (int)e->mul_rows, o.mul_tokens = e->mul_tokens, o.mul_at = e->mul_at;
    }
    o.act_a = e->act_a, o.act_b = e->act_b, o.act2 = e->act2;
    if (e->act2_from && e->act2_from < rows) o.act2_from = (int)e->act2_from;
    return 0;
}

int to_vec_in(const bitnet_hip_vector_input *in, size_t cols, VecIn &o) {
    BH_REQUIRE(in && in->x, "vector input: null pointer");
    BH_REQUIRE(in->kind >= BITNET_HIP_IN_PLAIN && in->kind <= BITNET_HIP_IN_RESIDUAL, "vector input: unknown kind %d", in->kind);
    if (in->kind != BITNET_HIP_IN_PLAIN) {
        if (in->kind == BITNET_HIP_IN_CONCAT)
            BH_REQUIRE(in->x2 && in->n > 0 && 2 * (size_t)in->n <= cols, "vector input: bad second half");
        else
            BH_REQUIRE((in->weight || in->kind == BITNET_HIP_IN_RESIDUAL) && in->n > 0 && (size_t)in->n <= cols && in->mean_n >= 0, "vector input: bad norm");
        if (in->kind >= BITNET_HIP_IN_RESIDUAL_NORM && in->y)
            BH_REQUIRE((in->post_weight || in->mult != 0.f) && (!in->x_out || (in->x_out != in->x && in->x_out != in->y)),
                       "vector input: the residual needs a norm or a factor, and a buffer of its own");
    }
    o.x = in->x, o.kind = in->kind, o.eps = in->eps, o.offset = in->weight_offset, o.weight = in->weight, o.y = in->y, o.post_weight = in->post_weight;
    o.scale = in->scale, o.gate = in->gate, o.x_out = in->y ? in->x_out : nullptr, o.n = in->n, o.mean_n = in->mean_n ? in->mean_n : in->n;
    o.mult = in->mult, o.center = in->center, o.bias = in->bias, o.x2 = in->x2, o.h_out = in->h_out, o.y_gate = in->y_gate;
    return 0;
}

int to_attn(const bitnet_hip_latent_attention *a, LatentAttn &o) {
    BH_REQUIRE(a && a->ccache && a->rcache && a->rope_cos && a->rope_sin, "latent attention: null pointer");
    BH_REQUIRE(a->heads > 0 && a->heads < 65536 && a->dimp % 32 == 0 && a->ldr % 32 == 0 && a->qd == a->dimp + a->ldr && a->vdimp > 0 && a->vdimp % 16 == 0 &&
                   a->ldc % 64 == 0 && a->kv_rank > 0 && a->kv_rank <= a->ldc && a->rot_dim <= a->ldr && a->rot_dim % 2 == 0 && a->capacity % 64 == 0 && (a->ldq == 0 || a->ldq >= a->heads * a->qd),
               "latent attention: bad shape");
    o.ldq = a->ldq ? a->ldq : a->heads * a->qd;
    o.ccache = a->ccache, o.rcache = a->rcache, o.ldc = (int)a->ldc, o.ldr = (int)a->ldr, o.kv_rank = (int)a->kv_rank, o.rot_dim = (int)a->rot_dim;
    o.heads = (int)a->heads, o.dimp = (int)a->dimp, o.qd = (int)a->qd, o.vdimp = (int)a->vdimp, o.scale = a->scale, o.sink = a->sink;
    o.rope_cos = a->rope_cos, o.rope_sin = a->rope_sin, o.capacity = (int)a->capacity;
    return 0;
}
}  // namespace

extern "C" {

int bitnet_hip_embed_bf16_dev(const uint16_t *table, size_t ld, const int32_t *tokens, const int32_t *offset, size_t n, size_t width, size_t vocab,
                              float scale, float *out, void *stream) {
    BH_GUARD_BEGIN
    BH_REQUIRE(table && tokens && out, "Null pointer passed to embed_bf16_dev");
    BH_REQUIRE(n > 0 && width > 0 && vocab > 0 && ld >= width, "embed_bf16: bad shape");
    BH_CHECK_DIMS(n, width);
    BH_HIP_TRY(launch_embed_bf16(table, ld, tokens, offset, (int)n, (int)width, (int)vocab, scale, nullptr, 0.f, TokenPairs(), out, (hipStream_t)stream));
    return BITNET_HIP_OK;
    BH_GUARD_END
}

int bitnet_hip_embed_pairs_bf16_dev(const uint16_t *table, size_t ld, const uint16_t *pairs, size_t ld_pairs, size_t buckets, uint64_t mul_prev, uint64_t mul_cur,
                                    const int32_t *tokens, const int32_t *offset, size_t n, size_t width, size_t vocab, float scale, float *out, void *stream) {
    BH_GUARD_BEGIN
    BH_REQUIRE(table && pairs && tokens && out, "Null pointer passed to embed_pairs_bf16_dev");
    BH_REQUIRE(n > 0 && width > 0 && vocab > 0 && ld >= width && ld_pairs >= width && buckets > 0 && mul_prev < (uint64_t(1) << 31) && mul_cur < (uint64_t(1) << 31),
               "embed_pairs_bf16: bad shape");
    BH_CHECK_DIMS(n, width);
    TokenPairs p;
    p.table = pairs, p.ld = ld_pairs, p.buckets = buckets, p.mul_prev = mul_prev, p.mul_cur = mul_cur;
    BH_HIP_TRY(launch_embed_bf16(table, ld, tokens, offset, (int)n, (int)width, (int)vocab, scale, nullptr, 0.f, p, out, (hipStream_t)stream));
    return BITNET_HIP_OK;
    BH_GUARD_END
}

int bitnet_hip_embed_norm_bf16_dev(const uint16_t *table, size_t ld, const int32_t *tokens, const int32_t *offset, size_t n, size_t width, size_t vocab,
                                   float scale, const float *norm_weight, float eps, float *out, void *stream) {
    BH_GUARD_BEGIN
    BH_REQUIRE(table && tokens && norm_weight && out, "Null pointer passed to embed_norm_bf16_dev");
    BH_REQUIRE(n > 0 && width > 0 && vocab > 0 && ld >= width, "embed_norm_bf16: bad shape");
    BH_CHECK_DIMS(n, width);
    BH_HIP_TRY(launch_embed_bf16(table, ld, tokens, offset, (int)n, (int)width, (int)vocab, scale, norm_weight, eps, TokenPairs(), out, (hipStream_t)stream));
    return BITNET_HIP_OK;
    BH_GUARD_END
}

int bitnet_hip_residual_norm_rows_dev(float *x, const float *y, size_t ldy, const float *post_weight, const float *scale, const float *next_weight,
                                      float weight_offset, float eps, size_t m, size_t width, void *h, size_t ldh, int h_f32, void *stream) {
    BH_GUARD_BEGIN
    BH_REQUIRE(x && (!y || (post_weight && ldy >= width)) && (!h || ldh >= width), "residual_norm_rows: bad arguments");
    BH_REQUIRE(m > 0 && width > 0, "residual_norm_rows: empty");
    BH_CHECK_DIMS(m, width);
    BH_HIP_TRY(launch_residual_norm_rows(x, y, ldy, post_weight, scale, next_weight, weight_offset, eps, (int)m, (int)width, h, ldh, h_f32,
                                         (hipStream_t)stream));
    return BITNET_HIP_OK;
    BH_GUARD_END
}

int bitnet_hip_gated_norm_rows_dev(const float *o, size_t ldo, const float *weight, const void *gate, size_t ldg, float eps, int gate_f32, size_t m,
                                   size_t n, size_t mean_n, void *h, size_t ldh, int h_f32, void *stream) {
    BH_GUARD_BEGIN
    BH_REQUIRE(o && weight && gate && h && m > 0 && n > 0 && mean_n > 0 && ldo >= n && ldg >= n && ldh >= n, "gated_norm_rows: bad arguments");
    BH_CHECK_DIMS(m, ldh);
    BH_HIP_TRY(launch_gated_norm_rows(o, ldo, weight, gate, ldg, gate_f32, eps, (int)m, (int)n, (int)mean_n, h, ldh, h_f32, (hipStream_t)stream));
    return BITNET_HIP_OK;
    BH_GUARD_END
}

int bitnet_hip_gather_rows_dev(const float *x, const int32_t *rows, size_t n, size_t width, float *out, void *stream) {
    BH_GUARD_BEGIN
    BH_REQUIRE(x && rows && out && n > 0 && width > 0, "gather_rows: bad arguments");
    BH_CHECK_DIMS(n, width);
    BH_HIP_TRY(launch_gather_rows(x, rows, (int)n, (int)width, out, (hipStream_t)stream));
    return BITNET_HIP_OK;
    BH_GUARD_END
}

int bitnet_hip_dense_matmul_dev(const void *a, size_t lda, int a_f32, const uint16_t *w, size_t ldw, const float *bias, size_t m, size_t n, size_t k,
                                int act0, int act1, size_t act_split, void *c, size_t ldc, int c_f32, size_t batch, size_t a_batch, size_t w_batch,
                                size_t c_batch, const bitnet_hip_epilogue *more, void *stream) {
    BH_GUARD_BEGIN
    BH_REQUIRE(a && w && c, "Null pointer passed to dense_matmul_dev");
    BH_REQUIRE(m > 0 && n > 0 && k > 0 && batch > 0 && batch < 65536, "dense_matmul: empty");
    const int gated = act0 & BITNET_HIP_ACT_GATED;
    act0 &= ~BITNET_HIP_ACT_GATED;
    BH_REQUIRE(k % 64 == 0 && lda >= k && ldw >= k && lda % 8 == 0 && ldw % 8 == 0 && ldc >= (gated ? n / 2 : n), "dense_matmul: k %zu must be a multiple of 64 inside lda %zu, ldw %zu; ldc %zu >= n %zu",
               k, lda, ldw, ldc, n);
    BH_REQUIRE(act_ok(act0) && act_ok(act1) && a_batch % 8 == 0 && w_batch % 8 == 0, "dense_matmul: bad activation or batch stride");
    BH_REQUIRE(!gated || (n % 2 == 0 && act0 != BITNET_HIP_ACT_XIELU && act_split == 0 && (a_f32 || !c_f32)), "dense_matmul: gated columns come in pairs, with one activation, in the activations' type");
    BH_CHECK_DIMS(m, lda);
    BH_CHECK_DIMS(n, ldw);
    BH_CHECK_DIMS(m, ldc);
    GemmArgsD g;
    if (int rc = to_epilogue(more, n, g.more)) return rc;
    BH_REQUIRE(!more || (!g.more.conv && more->pairs == 0 && more->act2_from == 0 && (!more->mul || (batch == 1 && !gated && (a_f32 || !c_f32)))),
               "dense_matmul: what a product of one row does, or a table of factors with pairs or f32 sums");
    g.a = a, g.w = w, g.bias = bias, g.c = c, g.m = (int)m, g.n = (int)n, g.k = (int)k, g.lda = lda, g.ldw = ldw, g.ldc = ldc;
    g.act0 = act0, g.act1 = act1, g.act_split = (int)act_split, g.gated = gated != 0, g.a_f32 = a_f32, g.c_f32 = c_f32;
    g.batch = (int)batch, g.a_batch = a_batch, g.w_batch = w_batch, g.c_batch = c_batch;
    BH_HIP_TRY(launch_dense_gemm(g, (hipStream_t)stream));
    return BITNET_HIP_OK;
    BH_GUARD_END
}

int bitnet_hip_latent_rows_dev(const bitnet_hip_latent_rows *rows, size_t m, int f32, void *stream) {
    BH_GUARD_BEGIN
    LatentRows r;
    if (int rc = to_latent_rows(rows, m, f32, r)) return rc;
    BH_CHECK_DIMS(m, rows->ldz);
    BH_HIP_TRY(launch_latent_rows(r, (hipStream_t)stream));
    return BITNET_HIP_OK;
    BH_GUARD_END
}

static int gemv_args(const bitnet_hip_vector_input *input, const uint16_t *w, size_t rows, size_t cols, size_t ld, float *y, GemvArgs &g) {
    BH_REQUIRE(w && y, "Null pointer passed to dense_gemv_dev");
    BH_REQUIRE(rows > 0 && cols >= 8 && cols % 8 == 0 && cols <= ld && ld % 8 == 0 && cols <= 38400 - 2560, "dense_gemv: bad shape %zu x %zu (ld %zu)", rows, cols, ld);
    BH_CHECK_DIMS(rows, ld);
    if (int rc = to_vec_in(input, cols, g.in)) return rc;
    g.w = w, g.rows = (int)rows, g.cols = (int)cols, g.ld = (int)ld, g.y = y;
    return 0;
}

int bitnet_hip_dense_gemv_dev(const bitnet_hip_vector_input *input, const uint16_t *w, size_t rows, size_t cols, size_t ld, const float *bias, int act0,
                              int act1, size_t act_split, float *y, size_t batch, size_t w_batch, size_t x_batch, size_t y_batch,
                              const bitnet_hip_latent_rows *latent, int latent_f32, const bitnet_hip_epilogue *more, void *stream) {
    BH_GUARD_BEGIN
    GemvArgs g;
    if (int rc = gemv_args(input, w, rows, cols, ld, y, g)) return rc;
    const int gated = act0 & BITNET_HIP_ACT_GATED;
    act0 &= ~BITNET_HIP_ACT_GATED;
    BH_REQUIRE(act_ok(act0) && act_ok(act1), "dense_gemv: unknown activation");
    if (int rc = to_epilogue(more, rows, g.more)) return rc;
    BH_REQUIRE(!gated || act0 != BITNET_HIP_ACT_XIELU, "dense_gemv: an activation with constants does not go with pairs");
    const size_t pairs = gated ? (more && more->pairs ? more->pairs : rows) : 0;
    BH_REQUIRE(!gated ? !more || more->pairs == 0 : pairs % 2 == 0 && (pairs < rows ? act_split >= pairs : act_split == 0), "dense_gemv: gated rows come in pairs, with one activation");
    BH_REQUIRE(batch > 0 && batch < 65536 && (batch == 1 || (g.in.kind == BITNET_HIP_IN_PLAIN && !g.more.conv && !g.more.mul && pairs == 0)) && w_batch % 8 == 0, "dense_gemv: bad batch");
    BH_CHECK_DIMS(batch, rows, ld);
    g.bias = bias, g.act0 = act0, g.act1 = act1, g.act_split = (int)act_split, g.gated = (int)pairs;
    g.batch = (int)batch, g.w_batch = w_batch, g.x_batch = x_batch, g.y_batch = y_batch;
    LatentRows r;
    if (latent) {
        if (int rc = to_latent_rows(latent, 1, latent_f32, r)) return rc;
        g.latent = &r;
    }
    BH_HIP_TRY(launch_dense_gemv(g, nullptr, (hipStream_t)stream));
    return BITNET_HIP_OK;
    BH_GUARD_END
}

int bitnet_hip_dense_logits_dev(const bitnet_hip_vector_input *input, const uint16_t *w, size_t vocab, size_t cols, size_t ld, float *logits,
                                void *scratch, int32_t *token, int32_t *pos, int32_t *history, const int32_t *n_forced, void *stream) {
    BH_GUARD_BEGIN
    GemvArgs g;
    BH_REQUIRE(scratch, "Null pointer passed to dense_logits_dev");
    if (int rc = gemv_args(input, w, vocab, cols, ld, logits, g)) return rc;
    g.best_val = static_cast<float *>(scratch);
    g.best_idx = reinterpret_cast<int *>(g.best_val + 1024);
    int n_wg = 0;
    BH_HIP_TRY(launch_dense_gemv(g, &n_wg, (hipStream_t)stream));
    if (token || pos) BH_HIP_TRY(launch_argmax_final(g.best_val, g.best_idx, n_wg, token, pos, history, n_forced, (hipStream_t)stream));
    return BITNET_HIP_OK;
    BH_GUARD_END
}

size_t bitnet_hip_latent_scratch_bytes(size_t heads, size_t ldc, size_t nq) { return latent_scratch_floats((int)heads, (int)ldc, (int)nq) * sizeof(float); }

int bitnet_hip_latent_decode_dev(const bitnet_hip_latent_attention *attn, const float *q, const float *qabs, const int32_t *pos, size_t q0, size_t nq,
                                 int f32, float *scratch, void *stream) {
    BH_GUARD_BEGIN
    LatentAttn a;
    if (int rc = to_attn(attn, a)) return rc;
    BH_REQUIRE(q && qabs && pos && scratch && nq > 0 && nq < 65536, "latent_decode: bad arguments");
    a.q = q, a.qabs = qabs, a.pos = pos, a.q0 = (int)q0, a.nq = (int)nq, a.f32 = f32, a.scratch = scratch;
    BH_HIP_TRY(launch_latent_decode(a, (hipStream_t)stream));
    return BITNET_HIP_OK;
    BH_GUARD_END
}

int bitnet_hip_latent_merge_dev(const bitnet_hip_latent_attention *attn, const uint16_t *uv, const int32_t *pos, size_t q0, size_t nq,
                                const float *scratch, void *out, size_t ldo, int out_bf16, void *stream) {
    BH_GUARD_BEGIN
    LatentAttn a;
    if (int rc = to_attn(attn, a)) return rc;
    BH_REQUIRE(uv && pos && scratch && out && nq > 0 && nq < 65536 && ldo >= attn->heads * attn->vdimp, "latent_merge: bad arguments");
    LatentMerge m;
    m.scratch = scratch, m.uv = uv, m.sink = a.sink, m.heads = a.heads, m.ldc = a.ldc, m.kv_rank = a.kv_rank, m.vdimp = a.vdimp;
    m.nq = (int)nq, m.q0 = (int)q0, m.pos = pos, m.out = out, m.ldo = ldo, m.out_bf16 = out_bf16;
    BH_HIP_TRY(launch_latent_merge(m, (hipStream_t)stream));
    return BITNET_HIP_OK;
    BH_GUARD_END
}

int bitnet_hip_latent_prefill_supported(size_t qd, size_t vdimp) { return qd <= 4096 && vdimp <= 4096 && latent_prefill_supported((int)qd, (int)vdimp) ? 1 : 0; }

int bitnet_hip_latent_prefill_dev(const bitnet_hip_latent_attention *attn, const uint16_t *q, const uint16_t *k, const uint16_t *vt, size_t ldvt,
                                  size_t n_ctx, size_t nq, uint16_t *out, size_t ldo, void *stream) {
    BH_GUARD_BEGIN
    LatentAttn a;
    if (int rc = to_attn(attn, a)) return rc;
    BH_REQUIRE(q && k && vt && out && nq > 0 && nq <= n_ctx && n_ctx <= attn->capacity && ldvt % 8 == 0 && ldvt >= (n_ctx + 63) / 64 * 64 &&
                   ldo >= attn->heads * attn->vdimp && ldo % 4 == 0 && attn->vdimp % 32 == 0,
               "latent_prefill: bad arguments");
    if (!latent_prefill_supported(a.qd, a.vdimp)) return set_error(BITNET_HIP_ERR_UNSUPPORTED, "latent_prefill: head of %d / %d columns", a.qd, a.vdimp);
    a.qb = q, a.k = k, a.vt = vt, a.ldvt = ldvt, a.n_ctx = (int)n_ctx, a.nq = (int)nq, a.out = out, a.ldo = ldo;
    BH_HIP_TRY(launch_latent_prefill(a, (hipStream_t)stream));
    return BITNET_HIP_OK;
    BH_GUARD_END
}

static int linear_args(const void *qkv, size_t ld, size_t n, size_t heads, size_t dimp, size_t vdimp, const float *decay_pow, float *state, float *out,
                       size_t ldo, LinearAttn &a) {
    BH_REQUIRE(qkv && decay_pow && state && out, "linear attention: null pointer");
    BH_REQUIRE(n > 0 && heads > 0 && heads < 65536 && dimp > 0 && vdimp > 0 && dimp <= 512 && vdimp <= 65536 && vdimp % 16 == 0 &&
                   ld >= heads * (2 * dimp + vdimp) && ldo >= heads * vdimp,
               "linear attention: bad shape (%zu heads of %zu / %zu)", heads, dimp, vdimp);
    BH_CHECK_DIMS(n, ld);
    a.qkv = qkv, a.ld = ld, a.n = (int)n, a.heads = (int)heads, a.dimp = (int)dimp, a.vdimp = (int)vdimp;
    a.decay_pow = decay_pow, a.state = state, a.out = out, a.ldo = ldo;
    return 0;
}

int bitnet_hip_linear_recurrent_dev(const float *qkv, size_t ld, size_t n, size_t heads, size_t dimp, size_t vdimp, const float *decay_pow,
                                    float *state, float *out, size_t ldo, void *stream) {
    BH_GUARD_BEGIN
    LinearAttn a;
    if (int rc = linear_args(qkv, ld, n, heads, dimp, vdimp, decay_pow, state, out, ldo, a)) return rc;
    BH_HIP_TRY(launch_linear_recurrent(a, (hipStream_t)stream));
    return BITNET_HIP_OK;
    BH_GUARD_END
}

size_t bitnet_hip_linear_workspace_bytes(size_t n, size_t heads, size_t dimp, size_t vdimp) {
    return linear_workspace_bytes((int)n, (int)heads, (int)dimp, (int)vdimp);
}

int bitnet_hip_linear_chunked_supported(size_t dimp, size_t vdimp) {
    return dimp <= 65536 && vdimp <= 65536 && linear_chunked_supported((int)dimp, (int)vdimp) ? 1 : 0;
}

int bitnet_hip_linear_chunked_dev(const uint16_t *qkv, size_t ld, size_t n, size_t heads, size_t dimp, size_t vdimp, const float *decay_pow,
                                  float *state, float *out, size_t ldo, void *workspace, size_t workspace_bytes, void *stream) {
    BH_GUARD_BEGIN
    LinearAttn a;
    if (int rc = linear_args(qkv, ld, n, heads, dimp, vdimp, decay_pow, state, out, ldo, a)) return rc;
    BH_REQUIRE(ld % 8 == 0 && ldo % 4 == 0 && workspace && workspace_bytes >= linear_workspace_bytes((int)n, (int)heads, (int)dimp, (int)vdimp),
               "linear_chunked: bad leading dimension or workspace");
    if (!linear_chunked_supported(a.dimp, a.vdimp)) return set_error(BITNET_HIP_ERR_UNSUPPORTED, "linear_chunked: head of %d / %d columns", a.dimp, a.vdimp);
    a.workspace = workspace, a.workspace_bytes = workspace_bytes;
    BH_HIP_TRY(launch_linear_chunked(a, (hipStream_t)stream));
    return BITNET_HIP_OK;
    BH_GUARD_END
}

}  // extern "C"
