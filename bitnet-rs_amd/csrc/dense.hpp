// dense.hpp -- device helpers and launcher declarations of the bf16-weight operators (kernels_dense.hip, kernels_experts.hip) and the
// sequence mixers (kernels_latent.hip, kernels_linear.hip, kernels_gqa.hip, kernels_delta.hip).
//
// Storage: weights bf16 row-major [rows][ld], ld a multiple of 64, columns past the matrix zero.  Activation matrices likewise
// have ld a multiple of 64; what lies past their columns must be FINITE (a weight's zero column cancels it).
#pragma once

#include "common.hpp"

namespace bitnet_hip {

typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));
typedef __bf16 bf16x4 __attribute__((ext_vector_type(4)));
typedef float f32x4 __attribute__((ext_vector_type(4)));
typedef uint32_t u32x4 __attribute__((ext_vector_type(4)));
typedef uint32_t u32x2 __attribute__((ext_vector_type(2)));

// ---- launch arguments ------------------------------------------------------------------------------------------------

// What else a product does with its rows (bitnet_hip_epilogue).
struct Epilogue {
    float act_a = 0.f, act_b = 0.f;
    int act2 = 0, act2_from = 0x7fffffff;
    int conv_from = 0, channels = 0, taps = 0;
    const float *conv = nullptr;
    float *ring = nullptr;
    const int *pos = nullptr;
    const uint16_t *mul = nullptr;
    size_t ld_mul = 0;
    int mul_rows = 0;
    const int *mul_tokens = nullptr, *mul_at = nullptr;
};

// How a matrix-vector product forms its input vector (bitnet_hip_vector_input).
struct VecIn {
    const float *x = nullptr;
    int kind = 0;                 // BITNET_HIP_IN_*
    float eps = 0.f, offset = 0.f;  // norm weight = offset + weight[i]
    const float *weight = nullptr;
    const float *y = nullptr, *post_weight = nullptr, *scale = nullptr;  // residual: x + scale * norm(y; post_weight)
    float *x_out = nullptr;
    const float *gate = nullptr;
    int n = 0, mean_n = 0;        // elements; what the mean divides by (padded heads hold zeros: fewer than n)
    float mult = 1.f;             // without post_weight: x + mult * y
    int center = 0;               // layer norm, with bias
    const float *bias = nullptr, *x2 = nullptr;
    float *h_out = nullptr;       // the vector formed
    const float *y_gate = nullptr;  // on what is added to x
};

struct GemvArgs {
    VecIn in;
    const uint16_t *w = nullptr;
    int rows = 0, cols = 0, ld = 0;  // cols: multiple of 8, <= ld
    int batch = 1;
    size_t w_batch = 0, x_batch = 0, y_batch = 0;  // elements between consecutive batch members
    const float *bias = nullptr;
    int act0 = 0, act1 = 0, act_split = 0;         // rows < act_split take act0, the others act1
    int gated = 0;                                 // rows 2 i and 2 i + 1 below this make element i: act0(row 2 i) * row 2 i + 1
    Epilogue more;
    float *y = nullptr;
    float *best_val = nullptr;                     // argmax partial per workgroup (batch 1)
    int *best_idx = nullptr;
    // extra work of the launch: the latent row of this position (see launch_latent_rows), one workgroup
    const struct LatentRows *latent = nullptr;
};

struct GemmArgsD {
    const void *a = nullptr;   // activations [m][lda]: bf16, or f32 with a_f32
    const uint16_t *w = nullptr;
    const float *bias = nullptr;
    void *c = nullptr;         // [m][ldc]
    int m = 0, n = 0, k = 0;   // k: multiple of 64, <= lda and ldw
    size_t lda = 0, ldw = 0, ldc = 0;
    int act0 = 0, act1 = 0, act_split = 0;
    int gated = 0;             // columns 2 i and 2 i + 1 make column i of c: act0(column 2 i) * column 2 i + 1 (n: columns ahead of that)
    int a_f32 = 0, c_f32 = 0;
    Epilogue more;
    int batch = 1;
    size_t a_batch = 0, w_batch = 0, c_batch = 0;
    // grouped form: the row tiles come from a list, (matrix, first row, rows) each; matrix i lies at w + i w_batch
    const int4 *tiles = nullptr;
    const int *n_tiles = nullptr;  // on the device
    int max_tiles = 0, tile = 0;
    const int *gather = nullptr;   // activation row of each row (nullptr: the row itself)
};

typedef bitnet_hip_sum_rows SumRows;
typedef bitnet_hip_gqa Gqa;
typedef bitnet_hip_delta Delta;
typedef bitnet_hip_experts_plan ExpertsPlan;
typedef bitnet_hip_router Router;

struct GqaStep {
    const float *row = nullptr;    // raw projections of the token
    const int *pos = nullptr;
    float *scratch = nullptr;
};

struct ExpertsUp {
    const float *logits = nullptr;
    Router r;
    const float *x = nullptr;
    const uint16_t *w = nullptr;
    int rows = 0, cols = 0, ld = 0, act = 0;
    int gated = 0;                 // rows 2 i and 2 i + 1 make column i
    float *y = nullptr;
    int ldy = 0;
    int *ids = nullptr;
    float *identity = nullptr;
};

struct ExpertsOut {
    const float *x0 = nullptr, *x1 = nullptr, *bias = nullptr;
    const uint16_t *w0 = nullptr, *w1 = nullptr;
    int cols0 = 0, ld0 = 0, cols1 = 0, ld1 = 0, ldx1 = 0, top = 0, rows = 0;
    const int *ids = nullptr;
    const float *identity = nullptr, *input = nullptr, *x0_scale = nullptr;
    float *y = nullptr;
};

// pairs of neighbouring tokens: the second table of an embedding (bitnet_hip_embed_pairs_bf16_dev)
struct TokenPairs {
    const uint16_t *table = nullptr;
    size_t ld = 0;
    uint64_t buckets = 0, mul_prev = 0, mul_cur = 0;
};

// rows of a down-projection output z -> normed query latent, normed key latent and rotated key part
struct LatentRows {
    const float *z = nullptr;      // [m][ldz]: [q_rank | kv_rank | rot_dim] (the last two absent when kv_rank == 0)
    int ldz = 0, q_rank = 0, kv_rank = 0, rot_dim = 0;
    const float *q_weight = nullptr, *kv_weight = nullptr;
    float eps = 0.f;
    void *cq = nullptr;            // [m][ldcq], nullable
    int ldcq = 0;
    void *ccache = nullptr;        // [capacity][ldc]
    void *rcache = nullptr;        // [capacity][ldr]
    int ldc = 0, ldr = 0;
    const float *rope_cos = nullptr, *rope_sin = nullptr;  // [capacity][rot_dim / 2]
    const int *pos = nullptr;      // first row's position
    int m = 0, f32 = 0;
};

struct LatentAttn {
    size_t ldq = 0;                // leading dimension of q, qb
    const float *q = nullptr;      // decode: f32 [nq][heads * qd] before rotation (the rotated part at [h * qd + dimp])
    const void *qb = nullptr;      // prompt: bf16 of the same
    const float *qabs = nullptr;   // decode: f32 [nq][heads * ldc] queries in latent space
    const void *ccache = nullptr, *rcache = nullptr;
    int ldc = 0, ldr = 0, kv_rank = 0, rot_dim = 0;
    int heads = 0, dimp = 0, qd = 0, vdimp = 0;
    float scale = 0.f;
    const float *sink = nullptr;
    const float *rope_cos = nullptr, *rope_sin = nullptr;
    const int *pos = nullptr;      // decode: query i stands at *pos + q0 + i
    int q0 = 0, nq = 0;
    int capacity = 0;
    int f32 = 0;
    float *scratch = nullptr;      // decode records
    // prompt
    const void *k = nullptr, *vt = nullptr;  // bf16 [n_ctx][heads * dimp], bf16 [heads * vdimp][ldvt]
    size_t ldvt = 0;
    int n_ctx = 0;
    void *out = nullptr;           // bf16 [nq][ldo]
    size_t ldo = 0;
};

struct LatentMerge {
    const float *scratch = nullptr;
    const uint16_t *uv = nullptr;  // [heads * vdimp][ldc]
    const float *sink = nullptr;
    int heads = 0, ldc = 0, kv_rank = 0, vdimp = 0, nq = 0, q0 = 0;
    const int *pos = nullptr;
    void *out = nullptr;           // [nq][ldo] f32 or bf16
    size_t ldo = 0;
    int out_bf16 = 0;
};

struct LinearAttn {
    const void *qkv = nullptr;     // [n][ld]: q [heads][dimp] | k [heads][dimp] | v [heads][vdimp]; f32 (recurrent), bf16 (chunked)
    size_t ld = 0;
    int n = 0, heads = 0, dimp = 0, vdimp = 0;
    const float *decay_pow = nullptr;  // [heads][kLinBlock + 1]: decay_h ^ i
    float *state = nullptr;        // [heads][vdimp][dimp]
    float *out = nullptr;          // [n][ldo]
    size_t ldo = 0;
    void *workspace = nullptr;     // chunked form
    size_t workspace_bytes = 0;
};

constexpr int kLinBlock = 128;     // tokens per block of the chunked linear attention
constexpr int kLatentTile = 64;    // keys per step of the decode attention
constexpr int kLatentSplits = 128;  // most records per (query, head)
constexpr int kLatentRecHead = 4;  // floats ahead of a record's vector: running maximum, sum, unused

constexpr int kGqaTile = 128;      // keys per workgroup and step of the decode attention
constexpr int kGqaSplits = 128;    // most records per (query, head, map)
constexpr int kMaxTaps = 64;       // of a convolution ahead of the attention
constexpr int kGqaRecHead = 4;     // floats ahead of a record's vector: running maximum (of base-2 scores), sum, unused
constexpr int kDeltaChunk = 64;    // tokens per chunk of the delta rule
constexpr int kDeltaUnits = 512;   // chunks x heads per pass over the workspace: one round of workgroups, and small enough to stay in the caches
constexpr int kMaxExperts = 1024, kMaxTop = 32;

hipError_t launch_embed_bf16(const uint16_t *table, size_t ld, const int *tokens, const int *offset, int n, int width, int vocab, float scale,
                             const float *norm_w, float eps, const TokenPairs &pairs, float *out, hipStream_t s);
hipError_t launch_conv_keep(const void *rows, size_t ld, int rows_f32, int channels, int taps, float *ring, const int *pos, int n, hipStream_t s);
hipError_t launch_sum_norm_rows(const SumRows &a, hipStream_t s);
hipError_t launch_residual_norm_rows(float *x, const float *y, size_t ldy, const float *post_w, const float *scale, const float *next_w,
                                     float offset, float eps, int m, int width, void *h, size_t ldh, int h_f32, hipStream_t s);
hipError_t launch_gated_norm_rows(const float *o, size_t ldo, const float *w, const void *gate, size_t ldg, int gate_f32, float eps, int m, int n,
                                  int mean_n, void *h, size_t ldh, int h_f32, hipStream_t s);
hipError_t launch_gather_rows(const float *x, const int *rows, int n, int width, float *out, hipStream_t s);
hipError_t launch_dense_gemv(const GemvArgs &a, int *n_wg_out, hipStream_t s);
hipError_t launch_dense_gemm(const GemmArgsD &a, hipStream_t s);
hipError_t launch_latent_rows(const LatentRows &a, hipStream_t s);
size_t latent_scratch_floats(int heads, int ldc, int nq);
bool latent_prefill_supported(int qd, int vdimp);
hipError_t launch_latent_decode(const LatentAttn &a, hipStream_t s);
hipError_t launch_latent_merge(const LatentMerge &a, hipStream_t s);
hipError_t launch_latent_prefill(const LatentAttn &a, hipStream_t s);
size_t linear_workspace_bytes(int n, int heads, int dimp, int vdimp);
bool linear_chunked_supported(int dimp, int vdimp);
hipError_t launch_linear_recurrent(const LinearAttn &a, hipStream_t s);
hipError_t launch_linear_chunked(const LinearAttn &a, hipStream_t s);
size_t gqa_scratch_floats(size_t heads, size_t maps, size_t vdimp, size_t nq);
bool gqa_supported(int dimp, int vdimp);
hipError_t launch_gqa_rows(const Gqa &g, void *rows, size_t ld, int rows_f32, int cache_f32, const int *pos, int n, void *q, size_t ldq, hipStream_t s);
hipError_t launch_gqa_step(const Gqa &g, const GqaStep &a, hipStream_t s);
hipError_t launch_gqa_any(const Gqa &g, const void *q, size_t ldq, int q_f32, int cache_f32, const int *pos, int q0, int nq, float *scratch, hipStream_t s);
hipError_t launch_gqa_merge(const Gqa &g, const int *pos, int q0, int nq, const float *scratch, void *out, size_t ldo, int out_bf16, hipStream_t s);
hipError_t launch_gqa_prefill(const Gqa &g, const uint16_t *q, size_t ldq, int n_ctx, int nq, uint16_t *out, size_t ldo, hipStream_t s);
bool delta_supported(int dimp, int vdimp);
bool delta_chunked_supported(int dimp, int vdimp);
size_t delta_workspace_bytes(size_t n, size_t heads, size_t dimp, size_t vdimp);
hipError_t launch_delta_step(const Delta &d, const float *row, const float *ba, const int *pos, float *out, hipStream_t s);
hipError_t launch_delta_rows(const Delta &d, const void *rows, size_t ld, int rows_f32, const float *ba, size_t ldba, const int *pos, int n, float *qk,
                             void *v, float *gates, hipStream_t s);
hipError_t launch_delta_recurrent(const Delta &d, const float *qk, const void *v, const float *gates, const void *rows, size_t ld, int rows_f32, int n,
                                  void *out, size_t ldo, hipStream_t s);
hipError_t launch_delta_chunked(const Delta &d, const float *qk, const uint16_t *v, const float *gates, const uint16_t *rows, size_t ld, int n,
                                uint16_t *out, size_t ldo, void *workspace, hipStream_t s);
hipError_t launch_experts_route(const float *logits, size_t ldz, const Router &r, const ExpertsPlan &p, hipStream_t s);
hipError_t launch_experts_up(const ExpertsUp &a, hipStream_t s);
hipError_t launch_experts_out(const ExpertsOut &a, hipStream_t s);

// ---- device helpers --------------------------------------------------------------------------------------------------

__device__ __forceinline__ float bf2f(uint32_t lo16) { return __builtin_bit_cast(float, lo16 << 16); }
__device__ __forceinline__ uint16_t f2bf(float v) { return __builtin_bit_cast(uint16_t, (__bf16)v); }
__device__ __forceinline__ float ld_act(const float *p, size_t i) { return p[i]; }
__device__ __forceinline__ float ld_act(const uint16_t *p, size_t i) { return bf2f(p[i]); }
__device__ __forceinline__ void st_act(float *p, size_t i, float v) { p[i] = v; }
__device__ __forceinline__ void st_act(uint16_t *p, size_t i, float v) { p[i] = f2bf(v); }

template <int CTRL>
__device__ __forceinline__ float dpp(float v) {
    return __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, v), CTRL, 0xf, 0xf, true));
}
// sum / maximum over the 16 lanes of a DPP row (every lane receives it)
__device__ __forceinline__ float row_sum(float v) {
    v += dpp<0x128>(v);
    v += dpp<0x124>(v);
    v += dpp<0x122>(v);
    return v + dpp<0x121>(v);
}
__device__ __forceinline__ float row_max(float v) {
    v = fmaxf(v, dpp<0x128>(v));
    v = fmaxf(v, dpp<0x124>(v));
    v = fmaxf(v, dpp<0x122>(v));
    return fmaxf(v, dpp<0x121>(v));
}
// The same over the four rows of a wave, lane by lane: with both operands holding the value, the swap leaves (rows 0, 0, 2, 2) and
// (1, 1, 3, 3), or (low half twice) and (high half twice).  As inline asm: hipcc (ROCm 7.2) folds the builtin's two results into one
// register when its operands are equal.
__device__ __forceinline__ void swap_rows16(float &a, float &b) { asm volatile("s_nop 1\n\tv_permlane16_swap_b32 %0, %1" : "+v"(a), "+v"(b)); }
__device__ __forceinline__ void swap_rows32(float &a, float &b) { asm volatile("s_nop 1\n\tv_permlane32_swap_b32 %0, %1" : "+v"(a), "+v"(b)); }
__device__ __forceinline__ float rows_sum(float v) {
    float w = v;
    swap_rows16(v, w);
    v += w;
    w = v;
    swap_rows32(v, w);
    return v + w;
}
__device__ __forceinline__ float rows_max(float v) {
    float w = v;
    swap_rows16(v, w);
    v = fmaxf(v, w);
    w = v;
    swap_rows32(v, w);
    return fmaxf(v, w);
}
__device__ __forceinline__ float wave_sum(float v) { return rows_sum(row_sum(v)); }

// sum over a workgroup of NW waves; slot: NW floats of LDS
template <int NW>
__device__ __forceinline__ float group_sum(float v, float *slot) {
    v = wave_sum(v);
    __syncthreads();
    if ((threadIdx.x & 63) == 0) slot[threadIdx.x >> 6] = v;
    __syncthreads();
    float t = slot[0];
#pragma unroll
    for (int i = 1; i < NW; ++i) t += slot[i];
    return t;
}

__device__ __forceinline__ float gelu_argument(float v) { return 0.7978845608028654f * (v + 0.044715f * v * v * v); }  // sqrt(2 / pi)
// BITNET_HIP_ACT_* without constants
__device__ __forceinline__ float activate(float v, int act) {
    switch (act) {
        case BITNET_HIP_ACT_SILU: return v / (1.0f + expf(-v));
        case BITNET_HIP_ACT_SIGMOID: return 1.0f / (1.0f + expf(-v));
        case BITNET_HIP_ACT_RELU2: {
            const float r = fmaxf(v, 0.0f);
            return r * r;
        }
        case BITNET_HIP_ACT_GELU_TANH: return v / (1.0f + expf(-2.0f * gelu_argument(v)));  // (1 + tanh z) / 2 = 1 / (1 + exp(-2 z))
        default: return v;
    }
}
// all of them
__device__ __forceinline__ float activate(float v, int act, float a, float b) {
    return act == BITNET_HIP_ACT_XIELU ? 0.5f * v + (v > 0.f ? a * v * v : b * (expm1f(v) - v)) : activate(v, act);
}

// a pair of floats as (high, low) bf16 pairs: high + low carries 16 of the 24 bits
__device__ __forceinline__ void split2(float a, float b, uint32_t &hi, uint32_t &lo) {
    const uint32_t ua = __builtin_bit_cast(uint32_t, a), ub = __builtin_bit_cast(uint32_t, b);
    const float la = a - __builtin_bit_cast(float, ua & 0xffff0000u), lb = b - __builtin_bit_cast(float, ub & 0xffff0000u);
    hi = __builtin_amdgcn_perm(ub, ua, 0x07060302u);
    lo = __builtin_amdgcn_perm(__builtin_bit_cast(uint32_t, lb), __builtin_bit_cast(uint32_t, la), 0x07060302u);
}

// eight floats as (high, low) fragments of the matrix cores
struct SplitFrag {
    bf16x8 hi, lo;
};
__device__ __forceinline__ SplitFrag split8(f32x4 a, f32x4 b) {
    u32x4 h, l;
    uint32_t x, y;
    split2(a.x, a.y, x, y), h.x = x, l.x = y;
    split2(a.z, a.w, x, y), h.y = x, l.y = y;
    split2(b.x, b.y, x, y), h.z = x, l.z = y;
    split2(b.z, b.w, x, y), h.w = x, l.w = y;
    return {__builtin_bit_cast(bf16x8, h), __builtin_bit_cast(bf16x8, l)};
}

__device__ __forceinline__ f32x4 mfma_bf16(bf16x8 a, bf16x8 b, f32x4 c) { return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, c, 0, 0, 0); }
// a product of two split operands (the low x low term is below the last bit kept)
__device__ __forceinline__ f32x4 mfma_split(const SplitFrag &a, const SplitFrag &b, f32x4 c) {
    c = mfma_bf16(a.hi, b.hi, c);
    c = mfma_bf16(a.hi, b.lo, c);
    return mfma_bf16(a.lo, b.hi, c);
}

}  // namespace bitnet_hip
