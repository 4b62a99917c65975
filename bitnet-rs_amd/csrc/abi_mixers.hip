// abi_mixers.hip -- section 5 of include/bitnet_hip.h, second part: rows of parallel blocks, grouped-head attention, the gated delta rule and
// mixture of experts.  Shapes are checked here against what the kernels assume; the kernels live in kernels_dense.hip, kernels_gqa.hip,
// kernels_delta.hip and kernels_experts.hip.
#include "dense.hpp"

using namespace bitnet_hip;

#define BH_REQUIRE(cond, ...)                                                      \
    do {                                                                           \
        if (!(cond)) return set_error(BITNET_HIP_ERR_INVALID_ARGUMENT, __VA_ARGS__); \
    } while (0)

namespace {
bool act_ok(int a) { return a >= BITNET_HIP_ACT_NONE && a <= BITNET_HIP_ACT_GELU_TANH; }  // (no constants here)

int check_gqa(const bitnet_hip_gqa *a) {
    BH_REQUIRE(a && a->q_factor && a->kcache && a->vcache, "gqa: null pointer");
    BH_REQUIRE(a->heads > 0 && a->heads < 32768 && a->kv_heads > 0 && a->heads % a->kv_heads == 0 && (a->maps == 1 || a->maps == 2) && a->dim > 0 &&
                   a->dim <= a->dimp && a->dimp % 32 == 0 && a->dimp <= 1024 && a->vdim > 0 && a->vdim <= a->vdimp && a->vdimp % 32 == 0 && a->vdimp <= 1024 &&
                   a->capacity > 0 && a->capacity % kGqaTile == 0,
               "gqa: bad shape (%zu heads on %zu, %zu maps of %zu in %zu, values %zu in %zu, capacity %zu)", a->heads, a->kv_heads, a->maps, a->dim, a->dimp,
               a->vdim, a->vdimp, a->capacity);
    BH_REQUIRE(a->rot_dims % 2 == 0 && a->rot_dims <= a->dim && (a->rot_dims == 0 || (a->rope_cos && a->rope_sin)), "gqa: bad rotation of %zu dimensions", a->rot_dims);
    BH_REQUIRE(a->chunk < (size_t(1) << 30) && (!a->sink || a->maps == 1) && (!a->values_are_keys || (a->maps == 1 && a->vdim == a->dim && a->vdimp == a->dimp)) &&
                   (!a->gate || a->ldgate >= (a->gate_columns ? a->heads * a->vdimp : a->heads)) && (!a->gate_columns || a->maps == 1),
               "gqa: bad chunk, sink, values or gate");
    BH_REQUIRE(a->window < (size_t(1) << 30) && !a->far_weight == !a->far_rate && (a->maps == 1 || (!a->far_weight && !a->queries_only)) && a->taps <= (size_t)kMaxTaps &&
                   (a->taps == 0 || (a->conv && a->ring)),
               "gqa: bad window, distance penalty, queries or convolution");
    BH_CHECK_DIMS(a->capacity, a->kv_heads * a->maps, a->dimp);
    BH_CHECK_DIMS(a->capacity, a->kv_heads, a->vdimp);
    return 0;
}
size_t gqa_row(const bitnet_hip_gqa *a) {
    return a->queries_only ? a->heads * a->dimp : (a->heads + a->kv_heads) * a->maps * a->dimp + (a->values_are_keys ? 0 : a->kv_heads * a->vdimp);
}

int check_delta(const bitnet_hip_delta *d) {
    BH_REQUIRE(d && d->conv && d->decay_rate && d->dt_bias && d->norm && d->state && d->ring, "delta: null pointer");
    BH_REQUIRE(d->heads > 0 && d->heads < 16384 && d->kv_heads > 0 && d->heads % d->kv_heads == 0 && d->dim > 0 && d->dim <= d->dimp && d->vdim > 0 &&
                   d->vdim <= d->vdimp && d->dimp <= 65536 && d->vdimp <= 65536 && delta_supported((int)d->dimp, (int)d->vdimp) && d->taps >= 1 && d->taps <= 64,
               "delta: bad shape (%zu heads on %zu, %zu in %zu, values %zu in %zu, %zu taps)", d->heads, d->kv_heads, d->dim, d->dimp, d->vdim, d->vdimp, d->taps);
    return 0;
}
size_t delta_row(const bitnet_hip_delta *d) { return 2 * d->kv_heads * d->dimp + 2 * d->heads * d->vdimp; }

int check_plan(const bitnet_hip_experts_plan *p) {
    BH_REQUIRE(p && p->counts && p->offsets && p->n_tiles && p->tiles && p->ids && p->slots && p->tokens && p->weights, "experts: no plan");
    BH_REQUIRE(p->m > 0 && p->experts > 0 && p->experts <= (size_t)kMaxExperts && p->top > 0 && p->top <= (size_t)kMaxTop && (p->tile == 64 || p->tile == 128),
               "experts: bad plan");
    BH_CHECK_DIMS(p->m, p->top);
    return 0;
}
int check_router(const bitnet_hip_router *r) {
    BH_REQUIRE(r && r->experts > 0 && r->experts <= (size_t)kMaxExperts && r->identity <= (size_t)kMaxExperts && r->experts + r->identity <= (size_t)kMaxExperts && r->top > 0 &&
                   r->top <= (size_t)kMaxTop && r->top <= r->experts + r->identity,
               "experts: bad router");
    BH_REQUIRE(r->groups == 0 || (r->identity == 0 && r->experts % r->groups == 0 && r->keep > 0 && r->keep <= r->groups && r->top <= r->keep * (r->experts / r->groups)),
               "experts: bad groups");
    return 0;
}
// tiles of a plan at most: every expert's last tile may be short
size_t plan_tiles(size_t m, size_t experts, size_t top, size_t tile) { return m * top / tile + experts; }
}  // namespace

extern "C" {

int bitnet_hip_sum_norm_rows_dev(const bitnet_hip_sum_rows *r, void *stream) {
    BH_GUARD_BEGIN
    BH_REQUIRE(r && r->x && r->m > 0 && r->width > 0 && (!r->y || r->ldy >= r->width), "sum_norm_rows: bad arguments");
    BH_REQUIRE(!r->h || (r->ldh >= (r->x2 ? 2 * r->width : r->width)), "sum_norm_rows: bad output");
    BH_REQUIRE(r->top == 0 || (r->expert_rows && r->slots && r->slot_weights && r->ld_expert >= r->width && (!r->input || r->ld_input >= r->width)),
               "sum_norm_rows: bad expert rows");
    BH_REQUIRE((!r->gate || r->ld_gate >= r->width) && (!r->y_scale || r->ld_y_scale > 0), "sum_norm_rows: bad gate or factors");
    BH_CHECK_DIMS(r->m, r->width);
    BH_HIP_TRY(launch_sum_norm_rows(*r, (hipStream_t)stream));
    return BITNET_HIP_OK;
    BH_GUARD_END
}

// ---- attention --------------------------------------------------------------------------------------------------------
size_t bitnet_hip_gqa_scratch_bytes(size_t heads, size_t maps, size_t vdimp, size_t nq) { return gqa_scratch_floats(heads, maps, vdimp, nq) * sizeof(float); }
int bitnet_hip_gqa_supported(size_t dimp, size_t vdimp) { return dimp <= 65536 && vdimp <= 65536 && gqa_supported((int)dimp, (int)vdimp) ? 1 : 0; }

int bitnet_hip_gqa_rows_dev(const bitnet_hip_gqa *a, void *rows, size_t ld, int rows_f32, int cache_f32, const int32_t *pos, size_t n, void *q, size_t ldq, void *stream) {
    BH_GUARD_BEGIN
    if (int rc = check_gqa(a)) return rc;
    if (!q) ldq = ld;
    BH_REQUIRE((q || a->taps == 0) && (!q || q != rows) && ldq >= a->heads * a->maps * a->dimp, "gqa_rows: bad place of the queries");
    BH_REQUIRE(rows && pos && n > 0 && n <= a->capacity && ld >= gqa_row(a) && (n == 1 || ld % 8 == 0) && (uintptr_t)rows % 16 == 0 && (rows_f32 || !cache_f32), "gqa_rows: bad arguments");
    BH_REQUIRE((a->heads + a->kv_heads) * a->maps + a->kv_heads * (a->vdimp / 32) < 65536, "gqa_rows: too many heads");
    BH_CHECK_DIMS(n, ld);
    BH_CHECK_DIMS(n, ldq);
    BH_HIP_TRY(launch_gqa_rows(*a, rows, ld, rows_f32, cache_f32, pos, (int)n, q ? q : rows, ldq, (hipStream_t)stream));
    return BITNET_HIP_OK;
    BH_GUARD_END
}

int bitnet_hip_conv_keep_dev(const void *rows, size_t ld, int rows_f32, size_t channels, size_t taps, float *ring, const int32_t *pos, size_t n, void *stream) {
    BH_GUARD_BEGIN
    BH_REQUIRE(rows && ring && pos && n > 0 && channels > 0 && ld >= channels && taps > 0 && taps <= (size_t)kMaxTaps, "conv_keep: bad arguments");
    BH_CHECK_DIMS(n, ld);
    BH_CHECK_DIMS(taps, channels);
    BH_HIP_TRY(launch_conv_keep(rows, ld, rows_f32, (int)channels, (int)taps, ring, pos, (int)n, (hipStream_t)stream));
    return BITNET_HIP_OK;
    BH_GUARD_END
}

int bitnet_hip_gqa_step_dev(const bitnet_hip_gqa *a, const float *row, const int32_t *pos, float *scratch, void *stream) {
    BH_GUARD_BEGIN
    if (int rc = check_gqa(a)) return rc;
    BH_REQUIRE(row && pos && scratch, "Null pointer passed to gqa_step_dev");
    if (!gqa_supported((int)a->dimp, (int)a->vdimp)) return set_error(BITNET_HIP_ERR_UNSUPPORTED, "gqa_step: head of %zu / %zu columns", a->dimp, a->vdimp);
    GqaStep s;
    s.row = row, s.pos = pos, s.scratch = scratch;
    BH_HIP_TRY(launch_gqa_step(*a, s, (hipStream_t)stream));
    return BITNET_HIP_OK;
    BH_GUARD_END
}

int bitnet_hip_gqa_any_dev(const bitnet_hip_gqa *a, const void *q, size_t ldq, int q_f32, int cache_f32, const int32_t *pos, size_t q0, size_t nq, float *scratch,
                           void *stream) {
    BH_GUARD_BEGIN
    if (int rc = check_gqa(a)) return rc;
    BH_REQUIRE(q && pos && scratch && nq > 0 && nq < 65536 && q0 < a->capacity && ldq >= a->heads * a->maps * a->dimp && (q_f32 || !cache_f32), "gqa_any: bad arguments");
    BH_HIP_TRY(launch_gqa_any(*a, q, ldq, q_f32, cache_f32, pos, (int)q0, (int)nq, scratch, (hipStream_t)stream));
    return BITNET_HIP_OK;
    BH_GUARD_END
}

int bitnet_hip_gqa_merge_dev(const bitnet_hip_gqa *a, const int32_t *pos, size_t q0, size_t nq, const float *scratch, void *out, size_t ldo, int out_bf16, void *stream) {
    BH_GUARD_BEGIN
    if (int rc = check_gqa(a)) return rc;
    BH_REQUIRE(pos && scratch && out && nq > 0 && nq < 65536 && q0 < a->capacity && ldo >= a->heads * a->vdimp, "gqa_merge: bad arguments");
    BH_HIP_TRY(launch_gqa_merge(*a, pos, (int)q0, (int)nq, scratch, out, ldo, out_bf16, (hipStream_t)stream));
    return BITNET_HIP_OK;
    BH_GUARD_END
}

int bitnet_hip_gqa_prefill_dev(const bitnet_hip_gqa *a, const uint16_t *q, size_t ldq, size_t n_ctx, size_t nq, uint16_t *out, size_t ldo, void *stream) {
    BH_GUARD_BEGIN
    if (int rc = check_gqa(a)) return rc;
    BH_REQUIRE(q && out && nq > 0 && nq <= n_ctx && n_ctx <= a->capacity && ldq % 8 == 0 && ldq >= a->heads * a->maps * a->dimp && ldo % 4 == 0 &&
                   ldo >= a->heads * a->vdimp,
               "gqa_prefill: bad arguments");
    BH_CHECK_DIMS(nq, ldq);
    if (!gqa_supported((int)a->dimp, (int)a->vdimp)) return set_error(BITNET_HIP_ERR_UNSUPPORTED, "gqa_prefill: head of %zu / %zu columns", a->dimp, a->vdimp);
    BH_HIP_TRY(launch_gqa_prefill(*a, q, ldq, (int)n_ctx, (int)nq, out, ldo, (hipStream_t)stream));
    return BITNET_HIP_OK;
    BH_GUARD_END
}

// ---- gated delta rule -------------------------------------------------------------------------------------------------
int bitnet_hip_delta_supported(size_t dimp, size_t vdimp) { return dimp <= 65536 && vdimp <= 65536 && delta_supported((int)dimp, (int)vdimp) ? 1 : 0; }
int bitnet_hip_delta_chunked_supported(size_t dimp, size_t vdimp) { return dimp <= 65536 && vdimp <= 65536 && delta_chunked_supported((int)dimp, (int)vdimp) ? 1 : 0; }

int bitnet_hip_delta_step_dev(const bitnet_hip_delta *d, const float *row, const float *ba, const int32_t *pos, float *out, void *stream) {
    BH_GUARD_BEGIN
    if (int rc = check_delta(d)) return rc;
    BH_REQUIRE(row && ba && pos && out, "Null pointer passed to delta_step_dev");
    BH_HIP_TRY(launch_delta_step(*d, row, ba, pos, out, (hipStream_t)stream));
    return BITNET_HIP_OK;
    BH_GUARD_END
}

int bitnet_hip_delta_rows_dev(const bitnet_hip_delta *d, const void *rows, size_t ld, int rows_f32, const float *ba, size_t ldba, const int32_t *pos, size_t n,
                              float *qk, void *v, float *gates, void *stream) {
    BH_GUARD_BEGIN
    if (int rc = check_delta(d)) return rc;
    BH_REQUIRE(rows && ba && pos && qk && v && gates && n > 0 && ld >= delta_row(d) && ld % 2 == 0 && ldba >= 2 * d->heads, "delta_rows: bad arguments");
    BH_CHECK_DIMS(n, ld);
    BH_HIP_TRY(launch_delta_rows(*d, rows, ld, rows_f32, ba, ldba, pos, (int)n, qk, v, gates, (hipStream_t)stream));
    return BITNET_HIP_OK;
    BH_GUARD_END
}

int bitnet_hip_delta_keep_dev(const bitnet_hip_delta *d, const void *rows, size_t ld, int rows_f32, const int32_t *pos, size_t n, void *stream) {
    BH_GUARD_BEGIN
    if (int rc = check_delta(d)) return rc;
    BH_REQUIRE(rows && pos && n > 0 && ld >= delta_row(d), "delta_keep: bad arguments");
    BH_CHECK_DIMS(n, ld);
    const size_t channels = 2 * d->kv_heads * d->dimp + d->heads * d->vdimp;
    BH_HIP_TRY(launch_conv_keep(rows, ld, rows_f32, (int)channels, (int)d->taps, d->ring, pos, (int)n, (hipStream_t)stream));
    return BITNET_HIP_OK;
    BH_GUARD_END
}

int bitnet_hip_delta_recurrent_dev(const bitnet_hip_delta *d, const float *qk, const void *v, const float *gates, const void *rows, size_t ld, int rows_f32,
                                   size_t n, void *out, size_t ldo, void *stream) {
    BH_GUARD_BEGIN
    if (int rc = check_delta(d)) return rc;
    BH_REQUIRE(qk && v && gates && rows && out && n > 0 && ld >= delta_row(d) && ldo >= d->heads * d->vdimp, "delta_recurrent: bad arguments");
    BH_CHECK_DIMS(n, ld);
    BH_HIP_TRY(launch_delta_recurrent(*d, qk, v, gates, rows, ld, rows_f32, (int)n, out, ldo, (hipStream_t)stream));
    return BITNET_HIP_OK;
    BH_GUARD_END
}

size_t bitnet_hip_delta_workspace_bytes(size_t n, size_t heads, size_t dimp, size_t vdimp) { return delta_workspace_bytes(n, heads, dimp, vdimp); }

int bitnet_hip_delta_chunked_dev(const bitnet_hip_delta *d, const float *qk, const uint16_t *v, const float *gates, const uint16_t *rows, size_t ld, size_t n,
                                 uint16_t *out, size_t ldo, void *workspace, size_t workspace_bytes, void *stream) {
    BH_GUARD_BEGIN
    if (int rc = check_delta(d)) return rc;
    BH_REQUIRE(qk && v && gates && rows && out && n > 0 && ld >= delta_row(d) && ld % 4 == 0 && ldo >= d->heads * d->vdimp && ldo % 4 == 0, "delta_chunked: bad arguments");
    BH_CHECK_DIMS(n, ld);
    if (!delta_chunked_supported((int)d->dimp, (int)d->vdimp)) return set_error(BITNET_HIP_ERR_UNSUPPORTED, "delta_chunked: head of %zu / %zu columns", d->dimp, d->vdimp);
    BH_REQUIRE(workspace && workspace_bytes >= delta_workspace_bytes(n, d->heads, d->dimp, d->vdimp), "delta_chunked: workspace too small");
    BH_HIP_TRY(launch_delta_chunked(*d, qk, v, gates, rows, ld, (int)n, out, ldo, workspace, (hipStream_t)stream));
    return BITNET_HIP_OK;
    BH_GUARD_END
}

// ---- experts ----------------------------------------------------------------------------------------------------------
// (the smaller tile needs the longer list: one size for both)
size_t bitnet_hip_experts_plan_bytes(size_t m, size_t experts, size_t top) {
    return (kMaxExperts + experts + 4 + 4 * plan_tiles(m, experts, top, 64) + 4 * m * top) * 4 + 64;
}

int bitnet_hip_experts_plan_make(void *workspace, size_t bytes, size_t m, size_t experts, size_t top, size_t tile, bitnet_hip_experts_plan *plan) {
    BH_GUARD_BEGIN
    BH_REQUIRE(workspace && plan && m > 0 && experts > 0 && experts <= (size_t)kMaxExperts && top > 0 && top <= (size_t)kMaxTop,
               "experts_plan: %zu of %zu experts (at most %d of %d)", top, experts, kMaxTop, kMaxExperts);
    BH_CHECK_DIMS(m, top);
    BH_REQUIRE((tile == 64 || tile == 128) && bytes >= bitnet_hip_experts_plan_bytes(m, experts, top) && (uintptr_t)workspace % 16 == 0, "experts_plan: bad workspace");
    int32_t *p = static_cast<int32_t *>(workspace);
    plan->m = m, plan->experts = experts, plan->top = top, plan->tile = tile, plan->max_tiles = plan_tiles(m, experts, top, tile);
    plan->counts = p, p += kMaxExperts;  // zero between uses, and at the same place whatever the sizes
    plan->tiles = p, p += 4 * plan_tiles(m, experts, top, 64);
    plan->offsets = p, p += experts;
    plan->n_tiles = p, p += 4;
    plan->ids = p, p += m * top;
    plan->slots = p, p += m * top;
    plan->tokens = p, p += m * top;
    plan->weights = reinterpret_cast<float *>(p);
    return BITNET_HIP_OK;
    BH_GUARD_END
}

int bitnet_hip_experts_route_dev(const float *logits, size_t ldz, const bitnet_hip_router *router, const bitnet_hip_experts_plan *plan, void *stream) {
    BH_GUARD_BEGIN
    if (int rc = check_plan(plan)) return rc;
    if (int rc = check_router(router)) return rc;
    BH_REQUIRE(logits && ldz >= router->experts + router->identity && plan->experts == router->experts && plan->top == router->top, "experts_route: bad arguments");
    BH_CHECK_DIMS(plan->m, ldz);
    BH_HIP_TRY(launch_experts_route(logits, ldz, *router, *plan, (hipStream_t)stream));
    return BITNET_HIP_OK;
    BH_GUARD_END
}

int bitnet_hip_experts_matmul_dev(const bitnet_hip_experts_plan *plan, int gather, const void *a, size_t lda, int a_f32, const uint16_t *w, size_t n, size_t k,
                                  size_t ldw, int act, void *c, size_t ldc, int c_f32, void *stream) {
    BH_GUARD_BEGIN
    if (int rc = check_plan(plan)) return rc;
    const int gated = act & BITNET_HIP_ACT_GATED;
    act &= ~BITNET_HIP_ACT_GATED;
    BH_REQUIRE(!gated || n % 2 == 0, "experts_matmul: gated columns come in pairs");
    BH_REQUIRE(a && w && c && n > 0 && k > 0 && k % 64 == 0 && lda >= k && ldw >= k && lda % 8 == 0 && ldw % 8 == 0 && ldc >= (gated ? n / 2 : n) && act_ok(act) && (a_f32 || !c_f32) &&
                   (!a_f32 || plan->tile == 64),
               "experts_matmul: bad arguments");
    BH_CHECK_DIMS(plan->experts, n, ldw);
    BH_CHECK_DIMS(plan->m * plan->top, ldc);
    // (a row's byte offset is a 32-bit number)
    BH_REQUIRE(!gather || a_f32 || plan->m * lda * 2 < (size_t(1) << 32), "experts_matmul: activations of 4 GiB or more");
    BH_CHECK_DIMS(plan->m * plan->top, lda);
    GemmArgsD g;
    g.a = a, g.w = w, g.c = c, g.m = (int)(plan->m * plan->top), g.n = (int)n, g.k = (int)k, g.lda = lda, g.ldw = ldw, g.ldc = ldc;
    g.act0 = g.act1 = act, g.gated = gated != 0, g.a_f32 = a_f32, g.c_f32 = c_f32, g.w_batch = n * ldw;
    g.tiles = reinterpret_cast<const int4 *>(plan->tiles), g.n_tiles = plan->n_tiles, g.max_tiles = (int)plan->max_tiles, g.tile = (int)plan->tile;
    g.gather = gather ? plan->tokens : nullptr;
    BH_HIP_TRY(launch_dense_gemm(g, (hipStream_t)stream));
    return BITNET_HIP_OK;
    BH_GUARD_END
}

int bitnet_hip_experts_up_dev(const float *logits, const bitnet_hip_router *router, const float *x, const uint16_t *w, size_t rows, size_t cols, size_t ld, int act,
                              float *y, size_t ldy, int32_t *ids, float *identity, void *stream) {
    BH_GUARD_BEGIN
    if (int rc = check_router(router)) return rc;
    const int gated = act & BITNET_HIP_ACT_GATED;
    act &= ~BITNET_HIP_ACT_GATED;
    BH_REQUIRE(logits && x && w && y && ids && rows > 0 && cols >= 8 && cols % 8 == 0 && cols <= ld && ld % 8 == 0 && cols <= 32768 && ldy >= (gated ? rows / 2 : rows) &&
                   act_ok(act) && (!gated || rows % 2 == 0) && (identity || router->identity == 0),
               "experts_up: bad arguments");
    BH_CHECK_DIMS(router->experts, rows, ld);
    ExpertsUp a;
    a.logits = logits, a.r = *router, a.x = x, a.w = w, a.rows = (int)rows, a.cols = (int)cols, a.ld = (int)ld;
    a.act = act, a.gated = gated != 0, a.y = y, a.ldy = (int)ldy, a.ids = ids, a.identity = identity;
    BH_HIP_TRY(launch_experts_up(a, (hipStream_t)stream));
    return BITNET_HIP_OK;
    BH_GUARD_END
}

int bitnet_hip_experts_out_dev(const float *x0, const uint16_t *w0, size_t cols0, size_t ld0, const float *bias, const float *x1, size_t ldx1, const uint16_t *w1,
                               size_t cols1, size_t ld1, const int32_t *ids, size_t top, size_t rows, const float *identity, const float *input, const float *x0_scale,
                               float *y, void *stream) {
    BH_GUARD_BEGIN
    if (!x0) w0 = nullptr, cols0 = ld0 = 0;
    BH_REQUIRE((!x0 || (w0 && cols0 >= 8)) && x1 && w1 && ids && y && top > 0 && top <= (size_t)kMaxTop && rows > 0 && cols0 % 8 == 0 && cols0 <= ld0 && ld0 % 8 == 0 &&
                   (!identity || input) && cols1 >= 8 && cols1 % 8 == 0 && cols1 <= ld1 && ld1 % 8 == 0 && ldx1 >= cols1,
               "experts_out: bad arguments");
    BH_CHECK_DIMS(rows, ld0);
    BH_CHECK_DIMS(rows, ld1);
    ExpertsOut a;
    a.x0 = x0, a.x1 = x1, a.bias = bias, a.w0 = w0, a.w1 = w1, a.cols0 = (int)cols0, a.ld0 = (int)ld0, a.cols1 = (int)cols1, a.ld1 = (int)ld1, a.ldx1 = (int)ldx1;
    a.top = (int)top, a.rows = (int)rows, a.ids = ids, a.identity = identity, a.input = input, a.x0_scale = x0_scale, a.y = y;
    const hipError_t e = launch_experts_out(a, (hipStream_t)stream);
    if (e == hipErrorInvalidValue) return set_error(BITNET_HIP_ERR_UNSUPPORTED, "experts_out: %zu + %zu x %zu columns do not fit a workgroup's memory", cols0, top, cols1);
    BH_HIP_TRY(e);
    return BITNET_HIP_OK;
    BH_GUARD_END
}

}  // extern "C"
