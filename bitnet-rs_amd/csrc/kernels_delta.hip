// kernels_delta.hip -- gated delta rule (gfx950): a state S [key][value] per head, carried from token to token in f32,
//   S <- g S;  u = beta (v - S^T k);  S <- S + k u^T;  o = S^T q,
// behind a short causal convolution with silu and unit norms of q and k, ahead of a norm per head and a gate.
//   k_delta_step       one token: convolution, norms, recurrence, output norm and gate in one launch
//   k_delta_rows       a portion's convolution, unit norms, decays and step sizes (its last inputs, for what follows: k_conv_keep)
//   k_delta_recurrent  those rows token by token
//   chunks of 64 tokens on the matrix cores: k_delta_chunk, k_delta_scan, k_delta_out
// With G_i the sum of log g up to token i of a chunk and L_ij = beta_i e^(G_i - G_j) k_i.k_j (j < i), the chunk's u satisfy
//   (I + L) U = diag(beta) V - diag(beta e^G) K S0,
// so with T = (I + L)^-1:  U = T diag(beta) V - (T diag(beta e^G) K) S0,  S' = e^G_end S0 + sum_j e^(G_end - G_j) k_j u_j^T,
//   o_i = e^G_i S0^T q_i + sum_{j <= i} e^(G_i - G_j) (k_j.q_i) u_j.
// k_delta_chunk forms T and the products with it for all chunks at once, k_delta_scan walks the chunks (one workgroup per 16 value columns,
// operands straight from memory in the order the matrix cores want them), k_delta_out forms the outputs of all chunks.
// f32 operands enter the matrix cores as (high, low) pairs of bf16 values; L and T are f32 throughout.
#include <algorithm>

#include "dense.hpp"

namespace bitnet_hip {

__device__ __forceinline__ float silu(float v) { return v / (1.0f + expf(-v)); }
__device__ __forceinline__ float softplus(float v) { return fmaxf(v, 0.f) + log1pf(expf(-fabsf(v))); }
__device__ __forceinline__ float log_decay(const Delta &p, int h, float a) { return -p.decay_rate[h] * softplus(a + p.dt_bias[h]); }

bool delta_supported(int dimp, int vdimp) { return dimp <= 256 && vdimp <= 256 && dimp % 32 == 0 && vdimp % 32 == 0; }
bool delta_chunked_supported(int dimp, int vdimp) { return delta_supported(dimp, vdimp) && dimp <= 128; }

// ---- token by token ---------------------------------------------------------------------------------------------------
// One workgroup per head.  Thread: value column tid % vdimp, keys tid / vdimp + SL j.
constexpr int kStepThreads = 1024;

struct StepLds {
    float q[256], k[256], v[256], u[256];
    float a[kStepThreads], b[kStepThreads];
    float slot[16];
};

// S and the output of one token from q, k, v in LDS; threads below vdimp return o
template <int NJ>
__device__ __forceinline__ float delta_token(StepLds &w, float (&s)[NJ], int dimp, int vdimp, int v, int sl, int SL, bool live, float g, float beta) {
    const int tid = threadIdx.x, lane = tid & 63;
    float a = 0.f, b = 0.f, kq = 0.f;
#pragma unroll
    for (int j = 0; j < NJ; ++j) {
        const int k = sl + SL * j;
        if (live && k < dimp) {
            a += s[j] * w.k[k];
            b += s[j] * w.q[k];
        }
    }
    for (int i = lane; i < dimp; i += 64) kq += w.k[i] * w.q[i];
    kq = wave_sum(kq);
    w.a[tid] = a, w.b[tid] = b;
    __syncthreads();
    float o = 0.f;
    if (tid < vdimp) {
        a = b = 0.f;
        for (int i = 0; i < SL; ++i) a += w.a[i * vdimp + tid], b += w.b[i * vdimp + tid];
        const float u = beta * (w.v[tid] - g * a);
        w.u[tid] = u;
        o = g * b + kq * u;
    }
    __syncthreads();
    if (live) {
        const float u = w.u[v];
#pragma unroll
        for (int j = 0; j < NJ; ++j)
            if (sl + SL * j < dimp) s[j] = g * s[j] + w.k[sl + SL * j] * u;
    }
    return o;
}

// sum over the threads below 256 (the others pass zero)
__device__ __forceinline__ float head_sum(float v, float *slot) {
    v = wave_sum(v);
    __syncthreads();
    if ((threadIdx.x & 63) == 0 && threadIdx.x < 256) slot[threadIdx.x >> 6] = v;
    __syncthreads();
    return (slot[0] + slot[1]) + (slot[2] + slot[3]);
}

template <int NJ>
__global__ __launch_bounds__(kStepThreads) void k_delta_step(Delta p, const float *row, const float *ba, const int *pos_ptr, float *out) {
    __shared__ StepLds w;
    const int tid = threadIdx.x, h = blockIdx.x, heads = (int)p.heads, kvh = (int)p.kv_heads, dimp = (int)p.dimp, vdimp = (int)p.vdimp, taps = (int)p.taps;
    const int per = heads / kvh, kv = h / per, C = 2 * kvh * dimp + heads * vdimp;
    const int SL = kStepThreads / vdimp, sl = tid / vdimp, v = tid - sl * vdimp;
    const bool live = sl < SL;
    float *st = p.state + (size_t)h * dimp * vdimp;
    float s[NJ];
#pragma unroll
    for (int j = 0; j < NJ; ++j) s[j] = live && sl + SL * j < dimp ? st[(size_t)(sl + SL * j) * vdimp + v] : 0.f;
    const int part = tid >> 8, c = tid & 255, pos = *pos_ptr;
    const int off = part == 0 ? kv * dimp + c : part == 1 ? (kvh + kv) * dimp + c : 2 * kvh * dimp + h * vdimp + c;
    const float gate = row[C + (size_t)h * vdimp + min(tid, vdimp - 1)], weight = p.norm[min(tid, vdimp - 1)], araw = ba[heads + h], braw = ba[h];
    float y = 0.f;
    if (part < 3 && c < (part == 2 ? vdimp : dimp)) {
        const float x = row[off];
        y = x * p.conv[(size_t)(taps - 1) * C + off];
        constexpr int AH = 4;  // earlier inputs in flight
        for (int j0 = 1; j0 < taps; j0 += AH) {
            float f[AH], in[AH];
#pragma unroll
            for (int e = 0; e < AH; ++e) {
                const int j = min(j0 + e, taps - 1);
                f[e] = p.conv[(size_t)(taps - 1 - j) * C + off];
                in[e] = p.ring[(size_t)((pos - j + taps) % taps) * C + off];
            }
#pragma unroll
            for (int e = 0; e < AH; ++e)
                if (j0 + e < taps && j0 + e <= pos) y += f[e] * in[e];
        }
        // (the slot written is none of those read: taps slots, taps - 1 earlier tokens)
        if (part == 2 || h == kv * per) p.ring[(size_t)(pos % taps) * C + off] = x;
        y = silu(y);
    }
    const float ss = wave_sum(part < 2 ? y * y : 0.f);
    if ((tid & 63) == 0 && part < 2) w.slot[tid >> 6] = ss;
    __syncthreads();
    if (part < 2) {
        const float *sum = w.slot + 4 * part;
        y *= 1.0f / sqrtf((sum[0] + sum[1]) + (sum[2] + sum[3]) + p.unit_eps);
        if (part == 0)
            w.q[c] = y * p.q_scale;
        else
            w.k[c] = y;
    } else if (part == 2) {
        w.v[c] = y;
    }
    const float g = expf(log_decay(p, h, araw)), beta = 1.0f / (1.0f + expf(-braw));
    __syncthreads();
    const float o = delta_token<NJ>(w, s, dimp, vdimp, v, sl, SL, live, g, beta);
#pragma unroll
    for (int j = 0; j < NJ; ++j)
        if (live && sl + SL * j < dimp) st[(size_t)(sl + SL * j) * vdimp + v] = s[j];
    const float inv = 1.0f / sqrtf(head_sum(o * o, w.slot) / (float)p.vdim + p.eps);
    if (tid < vdimp) out[(size_t)h * vdimp + tid] = o * inv * weight * silu(gate);
}

template <int NJ, class T>
__global__ __launch_bounds__(kStepThreads) void k_delta_recurrent(Delta p, const float *qk, const T *vr, const float *gates, const T *rows, size_t ld, int n, T *out,
                                                                  size_t ldo) {
    __shared__ StepLds w;
    const int tid = threadIdx.x, h = blockIdx.x, heads = (int)p.heads, kvh = (int)p.kv_heads, dimp = (int)p.dimp, vdimp = (int)p.vdimp;
    const int kv = h / (heads / kvh), C = 2 * kvh * dimp + heads * vdimp;
    const int SL = kStepThreads / vdimp, sl = tid / vdimp, v = tid - sl * vdimp;
    const bool live = sl < SL;
    float *st = p.state + (size_t)h * dimp * vdimp;
    float s[NJ];
#pragma unroll
    for (int j = 0; j < NJ; ++j) s[j] = live && sl + SL * j < dimp ? st[(size_t)(sl + SL * j) * vdimp + v] : 0.f;
    const int part = tid >> 8, c = tid & 255;
    for (int t = 0; t < n; ++t) {
        if (part < 2 && c < dimp) {
            const float x = qk[(size_t)t * 2 * kvh * dimp + (part * kvh + kv) * dimp + c];
            if (part == 0)
                w.q[c] = x;
            else
                w.k[c] = x;
        } else if (part == 2 && c < vdimp) {
            w.v[c] = ld_act(vr + (size_t)t * heads * vdimp, (size_t)h * vdimp + c);
        }
        const float g = expf(gates[(size_t)t * 2 * heads + h]), beta = gates[(size_t)t * 2 * heads + heads + h];
        __syncthreads();
        const float o = delta_token<NJ>(w, s, dimp, vdimp, v, sl, SL, live, g, beta);
        const float inv = 1.0f / sqrtf(head_sum(o * o, w.slot) / (float)p.vdim + p.eps);  // (its barriers also end this token's reads of q, k, v)
        if (tid < vdimp) st_act(out + (size_t)t * ldo, (size_t)h * vdimp + tid, o * inv * p.norm[tid] * silu(ld_act(rows + (size_t)t * ld, C + (size_t)h * vdimp + tid)));
    }
#pragma unroll
    for (int j = 0; j < NJ; ++j)
        if (live && sl + SL * j < dimp) st[(size_t)(sl + SL * j) * vdimp + v] = s[j];
}

// keys per thread
static int step_keys(const Delta &d) {
    const int SL = kStepThreads / (int)d.vdimp;
    return ((int)d.dimp + SL - 1) / SL;
}

hipError_t launch_delta_step(const Delta &d, const float *row, const float *ba, const int *pos, float *out, hipStream_t s) {
    if (!delta_supported((int)d.dimp, (int)d.vdimp)) return hipErrorInvalidValue;
    const int nj = step_keys(d);
    auto fn = nj <= 4 ? k_delta_step<4> : nj <= 16 ? k_delta_step<16> : nj <= 32 ? k_delta_step<32> : k_delta_step<64>;
    hipLaunchKernelGGL(fn, dim3(d.heads), dim3(kStepThreads), 0, s, d, row, ba, pos, out);
    return hipGetLastError();
}

hipError_t launch_delta_recurrent(const Delta &d, const float *qk, const void *v, const float *gates, const void *rows, size_t ld, int rows_f32, int n,
                                  void *out, size_t ldo, hipStream_t s) {
    if (!delta_supported((int)d.dimp, (int)d.vdimp)) return hipErrorInvalidValue;
    const int nj = step_keys(d);
    auto go = [&](auto fn, auto *vp, auto *rp, auto *op) { hipLaunchKernelGGL(fn, dim3(d.heads), dim3(kStepThreads), 0, s, d, qk, vp, gates, rp, ld, n, op, ldo); };
    if (rows_f32) {
        auto fn = nj <= 4 ? k_delta_recurrent<4, float> : nj <= 16 ? k_delta_recurrent<16, float> : nj <= 32 ? k_delta_recurrent<32, float> : k_delta_recurrent<64, float>;
        go(fn, (const float *)v, (const float *)rows, (float *)out);
    } else {
        auto fn = nj <= 16 ? k_delta_recurrent<16, uint16_t> : k_delta_recurrent<64, uint16_t>;
        go(fn, (const uint16_t *)v, (const uint16_t *)rows, (uint16_t *)out);
    }
    return hipGetLastError();
}

// ---- rows of a portion ------------------------------------------------------------------------------------------------
// A wave: one head's slice (q, k or v) of neighbouring tokens, two columns per lane and step; the window of earlier inputs moves along in
// registers.
constexpr int kRowTokens = 32, kRowTaps = 4;

__device__ __forceinline__ float2 ld2(const float *p, size_t i) { return *reinterpret_cast<const float2 *>(p + i); }
__device__ __forceinline__ void st2(float *p, size_t i, float2 v) { *reinterpret_cast<float2 *>(p + i) = v; }
__device__ __forceinline__ void st2(uint16_t *p, size_t i, float2 v) { *reinterpret_cast<uint32_t *>(p + i) = (uint32_t)f2bf(v.x) | (uint32_t)f2bf(v.y) << 16; }
__device__ __forceinline__ float2 ld2(const uint16_t *p, size_t i) {
    const uint32_t v = *reinterpret_cast<const uint32_t *>(p + i);
    return make_float2(bf2f(v & 0xffffu), __builtin_bit_cast(float, v & 0xffff0000u));
}

// TAPS: the convolution's taps, 0: more than kRowTaps
template <class T, int TAPS>
__global__ __launch_bounds__(256) void k_delta_rows(Delta p, const T *rows, size_t ld, const float *ba, size_t ldba, const int *pos_ptr, int n, float *qk, T *vo,
                                                    float *gates) {
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, y = blockIdx.y, pos0 = *pos_ptr;
    const int heads = (int)p.heads, kvh = (int)p.kv_heads, dimp = (int)p.dimp, vdimp = (int)p.vdimp, taps = TAPS ? TAPS : (int)p.taps, C = 2 * kvh * dimp + heads * vdimp;
    const bool value = y >= 2 * kvh;
    const int width = value ? vdimp : dimp, off = value ? 2 * kvh * dimp + (y - 2 * kvh) * vdimp : y * dimp;
    constexpr int PER = kRowTokens / 4, NT = TAPS ? TAPS : 1;
    const int t0 = blockIdx.x * kRowTokens + wave * PER, count = min(PER, n - t0);
    if (count <= 0) return;
    auto input = [&](int t, int col) {  // token t of the portion, or one ahead of it
        if (pos0 + t < 0) return make_float2(0.f, 0.f);
        return t >= 0 ? ld2(rows + (size_t)t * ld, col) : ld2(p.ring + (size_t)((pos0 + t) % taps) * C, col);
    };
    float2 x[PER][2];
#pragma unroll
    for (int c = 0; c < 2; ++c) {
        const int lc = lane * 2 + 128 * c, col = off + min(lc, width - 2);
        if (128 * c >= width) {
#pragma unroll
            for (int i = 0; i < PER; ++i) x[i][c] = make_float2(0.f, 0.f);
            continue;
        }
        if (TAPS) {
            float2 in[PER + NT - 1], f[NT];
#pragma unroll
            for (int j = 0; j < NT; ++j) f[j] = ld2(p.conv + (size_t)j * C, col);
#pragma unroll
            for (int i = 0; i < PER; ++i) in[NT - 1 + i] = ld2(rows + (size_t)min(t0 + i, n - 1) * ld, col);
#pragma unroll
            for (int j = 0; j < NT - 1; ++j) in[j] = input(t0 + j - (NT - 1), col);
#pragma unroll
            for (int i = 0; i < PER; ++i) {
                x[i][c] = make_float2(0.f, 0.f);
#pragma unroll
                for (int j = 0; j < NT; ++j) x[i][c].x += f[j].x * in[i + j].x, x[i][c].y += f[j].y * in[i + j].y;
            }
        } else {
            for (int i = 0; i < count; ++i) {
                float2 s = make_float2(0.f, 0.f);
                for (int j = 0; j < taps; ++j) {
                    const float2 f = ld2(p.conv + (size_t)(taps - 1 - j) * C, col), in = input(t0 + i - j, col);
                    s.x += f.x * in.x, s.y += f.y * in.y;
                }
#pragma unroll
                for (int k = 0; k < PER; ++k)
                    if (k == i) x[k][c] = s;
            }
        }
#pragma unroll
        for (int i = 0; i < PER; ++i) {
            const float live = lc < width ? 1.0f : 0.0f;
            x[i][c].x = live * silu(x[i][c].x), x[i][c].y = live * silu(x[i][c].y);
        }
    }
#pragma unroll
    for (int i = 0; i < PER; ++i) {
        if (i >= count) break;
        const int t = t0 + i;
        if (value) {
            T *dst = vo + (size_t)t * heads * vdimp + (size_t)(y - 2 * kvh) * vdimp;
#pragma unroll
            for (int c = 0; c < 2; ++c)
                if (lane * 2 + 128 * c < width) st2(dst, lane * 2 + 128 * c, x[i][c]);
        } else {
            const float ss = wave_sum((x[i][0].x * x[i][0].x + x[i][0].y * x[i][0].y) + (x[i][1].x * x[i][1].x + x[i][1].y * x[i][1].y));
            const float inv = 1.0f / sqrtf(ss + p.unit_eps) * (y < kvh ? p.q_scale : 1.0f);
            float *dst = qk + (size_t)t * 2 * kvh * dimp + (size_t)y * dimp;
#pragma unroll
            for (int c = 0; c < 2; ++c)
                if (lane * 2 + 128 * c < width) st2(dst, lane * 2 + 128 * c, make_float2(x[i][c].x * inv, x[i][c].y * inv));
        }
    }
    if (value && lane < count) {
        const int h = y - 2 * kvh, t = t0 + lane;
        gates[(size_t)t * 2 * heads + h] = log_decay(p, h, ba[(size_t)t * ldba + heads + h]);
        gates[(size_t)t * 2 * heads + heads + h] = 1.0f / (1.0f + expf(-ba[(size_t)t * ldba + h]));
    }
}

template <class T>
static void rows_go(const Delta &d, const T *rows, size_t ld, const float *ba, size_t ldba, const int *pos, int n, float *qk, T *v, float *gates, hipStream_t s) {
    const dim3 grid((n + kRowTokens - 1) / kRowTokens, 2 * d.kv_heads + d.heads);
    auto fn = d.taps == 1 ? k_delta_rows<T, 1> : d.taps == 2 ? k_delta_rows<T, 2> : d.taps == 3 ? k_delta_rows<T, 3> : d.taps == kRowTaps ? k_delta_rows<T, kRowTaps>
                                                                                                                               : k_delta_rows<T, 0>;
    hipLaunchKernelGGL(fn, grid, dim3(256), 0, s, d, rows, ld, ba, ldba, pos, n, qk, v, gates);
}

hipError_t launch_delta_rows(const Delta &d, const void *rows, size_t ld, int rows_f32, const float *ba, size_t ldba, const int *pos, int n, float *qk,
                             void *v, float *gates, hipStream_t s) {
    if (rows_f32)
        rows_go(d, (const float *)rows, ld, ba, ldba, pos, n, qk, (float *)v, gates, s);
    else
        rows_go(d, (const uint16_t *)rows, ld, ba, ldba, pos, n, qk, (uint16_t *)v, gates, s);
    return hipGetLastError();
}

// ---- chunks -----------------------------------------------------------------------------------------------------------
// Fragments lie in memory as the matrix cores take them: 64 lanes x 16 bytes, the high half ahead of the low half.  Contractions over key
// columns or tokens that meet a product's own accumulators go in their order: element e of lane group g is index 4 g + e of the first 16-row
// tile (e < 4) or 4 g + e - 4 of the second.
struct DeltaWs {
    u32x4 *w;   // [chunk][4 token tiles][nk][2][64]   -(T diag(beta e^G) K), rows = tokens, contraction = key columns
    u32x4 *k;   // [chunk][2 nk key tiles][2][2][64]   e^(G_end - G) K transposed, rows = key columns, contraction = tokens
    f32x4 *ut;  // [chunk][nv value tiles][4 token tiles][64]  T diag(beta) V as accumulators
    u32x4 *s;   // [chunk][nv][nk][2][64]              the state ahead of the chunk, contraction = key columns
    u32x4 *u;   // [chunk][nv][2][2][64]               U, contraction = tokens
    float *g;   // [chunk][64]                         G
    int nc, nk, nv;  // chunks; 32-column steps of a key; 16-column tiles of a value
};
constexpr int kTriStride = 68;

__device__ __forceinline__ f32x4 mfma_f32(float a, float b, f32x4 c) { return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0); }
__device__ __forceinline__ SplitFrag frag_at(const float *p) { return split8(*reinterpret_cast<const f32x4 *>(p), *reinterpret_cast<const f32x4 *>(p + 4)); }

__global__ __launch_bounds__(256, 2) void k_delta_chunk(Delta p, const float *qk, const uint16_t *vr, const float *gates, int n, DeltaWs w) {
    extern __shared__ __attribute__((aligned(16))) float lds[];
    __shared__ float sG[64], sB[64], sE[64], sF[64];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, r16 = lane & 15, g = lane >> 4;
    const int c = blockIdx.x, h = blockIdx.y, heads = (int)p.heads, kvh = (int)p.kv_heads, dimp = (int)p.dimp, vdimp = (int)p.vdimp, kv = h / (heads / kvh);
    const int t0 = c * kDeltaChunk, len = min(kDeltaChunk, n - t0), KS = dimp + 4;
    const size_t ch = (size_t)h * w.nc + c;
    float *lk = lds, *lL = lk + 64 * KS, *lT = lL + 64 * kTriStride;
    const float *K = qk + (size_t)t0 * 2 * kvh * dimp + (size_t)(kvh + kv) * dimp;
    for (int i = tid; i < 64 * (dimp / 4); i += 256) {
        const int t = i / (dimp / 4), d = (i - t * (dimp / 4)) * 4;
        f32x4 v = *reinterpret_cast<const f32x4 *>(K + (size_t)min(t, len - 1) * 2 * kvh * dimp + d);
        *reinterpret_cast<f32x4 *>(lk + t * KS + d) = t < len ? v : f32x4{0.f, 0.f, 0.f, 0.f};
    }
    for (int i = tid; i < 64 * kTriStride; i += 256) lT[i] = 0.f;
    if (wave == 0) {
        const float *gt = gates + (size_t)(t0 + min(lane, len - 1)) * 2 * heads + h;
        float G = lane < len ? gt[0] : 0.f;
        const float beta = lane < len ? gt[heads] : 0.f;
#pragma unroll
        for (int off = 1; off < 64; off <<= 1) {
            const float o = __shfl_up(G, off, 64);
            if (lane >= off) G += o;
        }
        const float end = __shfl(G, 63, 64);
        sG[lane] = G, sB[lane] = beta, sE[lane] = beta * expf(G), sF[lane] = expf(end - G);
        w.g[ch * 64 + lane] = G;
    }
    __syncthreads();
    {  // L: row tile = wave
        SplitFrag a[4];
#pragma unroll
        for (int kk = 0; kk < 4; ++kk)
            if (kk < w.nk) a[kk] = frag_at(lk + (wave * 16 + r16) * KS + kk * 32 + g * 8);
        for (int jt = 0; jt <= wave; ++jt) {
            f32x4 d = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int kk = 0; kk < 4; ++kk)
                if (kk < w.nk) d = mfma_split(a[kk], frag_at(lk + (jt * 16 + r16) * KS + kk * 32 + g * 8), d);
            const int j = jt * 16 + r16;
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                const int i = wave * 16 + g * 4 + e;
                lL[i * kTriStride + j] = j < i ? sB[i] * expf(sG[i] - sG[j]) * d[e] : 0.f;
            }
        }
    }
    __syncthreads();
    {  // diagonal blocks of T: a lane solves one column (the four lane groups alike)
        const float *L = lL + wave * 16 * kTriStride + wave * 16;
        float x[16];
#pragma unroll
        for (int i = 0; i < 16; ++i) {
            x[i] = i == r16 ? 1.0f : 0.0f;
#pragma unroll
            for (int k = 0; k < i; ++k) x[i] -= L[i * kTriStride + k] * x[k];
        }
        if (g == 0)
#pragma unroll
            for (int i = 0; i < 16; ++i) lT[(wave * 16 + i) * kTriStride + wave * 16 + r16] = x[i];
    }
    __syncthreads();
    // below the diagonal: block column = wave, T_ij = -T_ii sum_k L_ik T_kj
    for (int it = wave + 1; it < 4; ++it) {
        f32x4 m = f32x4{0.f, 0.f, 0.f, 0.f};
        for (int kt = wave; kt < it; ++kt)
#pragma unroll
            for (int s = 0; s < 4; ++s)
                m = mfma_f32(lL[(it * 16 + r16) * kTriStride + kt * 16 + s * 4 + g], lT[(kt * 16 + s * 4 + g) * kTriStride + wave * 16 + r16], m);
        float *dst = lT + it * 16 * kTriStride + wave * 16;
#pragma unroll
        for (int e = 0; e < 4; ++e) dst[(g * 4 + e) * kTriStride + r16] = m[e];
        f32x4 r = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int s = 0; s < 4; ++s) r = mfma_f32(lT[(it * 16 + r16) * kTriStride + it * 16 + s * 4 + g], dst[(s * 4 + g) * kTriStride + r16], r);
#pragma unroll
        for (int e = 0; e < 4; ++e) dst[(g * 4 + e) * kTriStride + r16] = -r[e];
    }
    __syncthreads();
    auto put = [&](u32x4 *dst, const SplitFrag &f) {
        dst[lane] = __builtin_bit_cast(u32x4, f.hi);
        dst[64 + lane] = __builtin_bit_cast(u32x4, f.lo);
    };
    for (int kk = wave; kk < w.nk; kk += 4) {
        SplitFrag a[2][2];
#pragma unroll
        for (int dt = 0; dt < 2; ++dt)
#pragma unroll
            for (int k2 = 0; k2 < 2; ++k2) {
                f32x4 x, y;
                const float *col = lk + (kk * 2 + dt) * 16 + r16;
                // decayed keys for the state, in the order of U's accumulators
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    const int ta = k2 * 32 + g * 4 + e, tb = ta + 16;
                    x[e] = col[ta * KS] * sF[ta], y[e] = col[tb * KS] * sF[tb];
                }
                put(w.k + (((ch * 2 * w.nk + kk * 2 + dt) * 2 + k2) * 2) * 64, split8(x, y));
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    const int ta = k2 * 32 + g * 8 + e, tb = ta + 4;
                    x[e] = col[ta * KS] * sE[ta], y[e] = col[tb * KS] * sE[tb];
                }
                a[dt][k2] = split8(x, y);
            }
#pragma unroll
        for (int it = 0; it < 4; ++it) {
            f32x4 d[2] = {f32x4{0.f, 0.f, 0.f, 0.f}, f32x4{0.f, 0.f, 0.f, 0.f}};
#pragma unroll
            for (int k2 = 0; k2 <= it / 2; ++k2) {
                const SplitFrag b = frag_at(lT + (it * 16 + r16) * kTriStride + k2 * 32 + g * 8);
#pragma unroll
                for (int dt = 0; dt < 2; ++dt) d[dt] = mfma_split(a[dt][k2], b, d[dt]);
            }
            put(w.w + (((ch * 4 + it) * w.nk + kk) * 2) * 64, split8(-d[0], -d[1]));
        }
    }
    const uint16_t *V = vr + (size_t)t0 * heads * vdimp + (size_t)h * vdimp;
    for (int vt = wave; vt < w.nv; vt += 4) {
        SplitFrag b[2];
#pragma unroll
        for (int k2 = 0; k2 < 2; ++k2) {
            f32x4 x, y;
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                const int ta = k2 * 32 + g * 8 + e, tb = ta + 4;
                x[e] = bf2f(V[(size_t)min(ta, len - 1) * heads * vdimp + vt * 16 + r16]) * sB[ta];  // (beta is zero past the end)
                y[e] = bf2f(V[(size_t)min(tb, len - 1) * heads * vdimp + vt * 16 + r16]) * sB[tb];
            }
            b[k2] = split8(x, y);
        }
#pragma unroll
        for (int it = 0; it < 4; ++it) {
            f32x4 d = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int k2 = 0; k2 <= it / 2; ++k2) d = mfma_split(frag_at(lT + (it * 16 + r16) * kTriStride + k2 * 32 + g * 8), b[k2], d);
            w.ut[((ch * w.nv + vt) * 4 + it) * 64 + lane] = d;
        }
    }
}

// One workgroup: one head, 16 value columns.  Wave w takes token tile w of U and key tiles 2 w, 2 w + 1 of the state; state and U meet in LDS as
// fragments, twice per chunk.  Operands come straight from memory, requested two chunks ahead.
template <int NK>
__global__ __launch_bounds__(256, 1) void k_delta_scan(Delta p, DeltaWs w) {
    __shared__ u32x4 ss[NK][2][64], su[2][2][64];
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), r16 = lane & 15, g = lane >> 4;
    // consecutive workgroups go to the eight XCDs in turn: a head's value tiles stay on one of them, whose L2 then holds its operands
    const int x = blockIdx.x & 7, rest = blockIdx.x >> 3, h = (rest / w.nv) * 8 + x, vt = rest % w.nv;
    if (h >= (int)p.heads) return;
    // (waves past the state's tiles repeat the last ones, stores included: no store stands behind a branch, which would keep hipcc from counting
    // the loads in flight)
    const int vdimp = (int)p.vdimp, kt = min(wave, NK - 1);
    float *st = p.state + (size_t)h * p.dimp * vdimp + vt * 16 + r16;
    f32x4 s[2];
#pragma unroll
    for (int d = 0; d < 2; ++d)
#pragma unroll
        for (int e = 0; e < 4; ++e) s[d][e] = st[(size_t)((2 * kt + d) * 16 + g * 4 + e) * vdimp];
    u32x4 wf[2][NK][2], kf[2][2][2][2];
    f32x4 ut[2];
    float ge[2];
    auto fetch_w = [&](int b, int c) {
        const size_t ch = (size_t)h * w.nc + min(c, w.nc - 1);
#pragma unroll
        for (int kk = 0; kk < NK; ++kk)
#pragma unroll
            for (int e = 0; e < 2; ++e) wf[b][kk][e] = w.w[(((ch * 4 + wave) * NK + kk) * 2 + e) * 64 + lane];
        ut[b] = w.ut[((ch * w.nv + vt) * 4 + wave) * 64 + lane];
    };
    auto fetch_k = [&](int b, int c) {
        const size_t ch = (size_t)h * w.nc + min(c, w.nc - 1);
#pragma unroll
        for (int d = 0; d < 2; ++d)
#pragma unroll
            for (int k2 = 0; k2 < 2; ++k2)
#pragma unroll
                for (int e = 0; e < 2; ++e) kf[b][d][k2][e] = w.k[(((ch * 2 * NK + 2 * kt + d) * 2 + k2) * 2 + e) * 64 + lane];
        ge[b] = w.g[ch * 64 + 63];
    };
    auto chunk = [&](int b, int c) {
        const size_t ch = (size_t)h * w.nc + c;
        {
            const SplitFrag f = split8(s[0], s[1]);
            ss[kt][0][lane] = __builtin_bit_cast(u32x4, f.hi);
            ss[kt][1][lane] = __builtin_bit_cast(u32x4, f.lo);
            u32x4 *dst = w.s + (((ch * w.nv + vt) * NK + kt) * 2) * 64 + lane;
            dst[0] = __builtin_bit_cast(u32x4, f.hi);
            dst[64] = __builtin_bit_cast(u32x4, f.lo);
        }
        __syncthreads();
        f32x4 a[3] = {ut[b], f32x4{0.f, 0.f, 0.f, 0.f}, f32x4{0.f, 0.f, 0.f, 0.f}};
        u32x4 sf[NK][2];
#pragma unroll
        for (int kk = 0; kk < NK; ++kk) sf[kk][0] = ss[kk][0][lane], sf[kk][1] = ss[kk][1][lane];
        __builtin_amdgcn_sched_barrier(0);
#pragma unroll
        for (int kk = 0; kk < NK; ++kk) {
            const bf16x8 hi = __builtin_bit_cast(bf16x8, sf[kk][0]), lo = __builtin_bit_cast(bf16x8, sf[kk][1]);
            a[0] = mfma_bf16(__builtin_bit_cast(bf16x8, wf[b][kk][0]), hi, a[0]);
            a[1] = mfma_bf16(__builtin_bit_cast(bf16x8, wf[b][kk][0]), lo, a[1]);
            a[2] = mfma_bf16(__builtin_bit_cast(bf16x8, wf[b][kk][1]), hi, a[2]);
        }
        const f32x4 u = a[0] + (a[1] + a[2]);
        {
            uint32_t h0, l0, h1, l1;
            split2(u.x, u.y, h0, l0);
            split2(u.z, u.w, h1, l1);
            reinterpret_cast<u32x2 *>(&su[wave >> 1][0][lane])[wave & 1] = u32x2{h0, h1};
            reinterpret_cast<u32x2 *>(&su[wave >> 1][1][lane])[wave & 1] = u32x2{l0, l1};
        }
        __builtin_amdgcn_sched_barrier(0);
        fetch_w(b, c + 2);
        __syncthreads();
        const u32x4 uf[2][2] = {{su[0][0][lane], su[0][1][lane]}, {su[1][0][lane], su[1][1][lane]}};
        w.u[(((ch * w.nv + vt) * 2 + (wave >> 1)) * 2 + (wave & 1)) * 64 + lane] = su[wave >> 1][wave & 1][lane];
        __builtin_amdgcn_sched_barrier(0);
        const float end = expf(ge[b]);
        f32x4 d0[2], d1[2];
#pragma unroll
        for (int d = 0; d < 2; ++d) d0[d] = s[d] * end, d1[d] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int k2 = 0; k2 < 2; ++k2) {
            const bf16x8 hi = __builtin_bit_cast(bf16x8, uf[k2][0]), lo = __builtin_bit_cast(bf16x8, uf[k2][1]);
#pragma unroll
            for (int d = 0; d < 2; ++d) {
                d0[d] = mfma_bf16(__builtin_bit_cast(bf16x8, kf[b][d][k2][0]), hi, d0[d]);
                d1[d] = mfma_bf16(__builtin_bit_cast(bf16x8, kf[b][d][k2][0]), lo, d1[d]);
            }
#pragma unroll
            for (int d = 0; d < 2; ++d) d1[d] = mfma_bf16(__builtin_bit_cast(bf16x8, kf[b][d][k2][1]), hi, d1[d]);
        }
#pragma unroll
        for (int d = 0; d < 2; ++d) s[d] = d0[d] + d1[d];
        __builtin_amdgcn_sched_barrier(0);
        fetch_k(b, c + 2);
    };
    fetch_w(0, 0), fetch_k(0, 0), fetch_w(1, 1), fetch_k(1, 1);
    int c = 0;
    for (; c + 1 < w.nc; c += 2) {
        chunk(0, c);
        chunk(1, c + 1);
    }
    if (c < w.nc) chunk(0, c);
#pragma unroll
    for (int d = 0; d < 2; ++d)
#pragma unroll
        for (int e = 0; e < 4; ++e) st[(size_t)((2 * kt + d) * 16 + g * 4 + e) * vdimp] = s[d][e];
}

// Outputs of a chunk and head, two waves of two token tiles each (the first and the last, the two between): O^T = S^T Q^T and U^T P^T, then norm
// and gate.  A value tile's operands are requested one tile ahead.
template <int NK, int NV>
__global__ __launch_bounds__(128, NV > 8 ? 1 : 2) void k_delta_out(Delta p, const float *qk, const uint16_t *rows, size_t ld, int n, DeltaWs w, uint16_t *out, size_t ldo) {
    __shared__ float sG[64];
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), r16 = lane & 15, g = lane >> 4;
    const int c = blockIdx.x, h = blockIdx.y, heads = (int)p.heads, kvh = (int)p.kv_heads, dimp = (int)p.dimp, vdimp = (int)p.vdimp, kv = h / (heads / kvh);
    const int t0 = c * kDeltaChunk, len = min(kDeltaChunk, n - t0), C = 2 * kvh * dimp + heads * vdimp;
    const size_t ch = (size_t)h * w.nc + c, ldq = (size_t)2 * kvh * dimp;
    if (tid < 64) sG[tid] = w.g[ch * 64 + tid];
    __syncthreads();
    if (wave * 16 >= len) return;
    const float *Q = qk + (size_t)t0 * ldq + (size_t)kv * dimp, *K = Q + (size_t)kvh * dimp;
    auto load = [&](const float *m, int t, int kk) {
        const float *src = m + (size_t)min(t, len - 1) * ldq + kk * 32 + g * 4;
        return split8(*reinterpret_cast<const f32x4 *>(src), *reinterpret_cast<const f32x4 *>(src + 16));
    };
    const int tile[2] = {wave, 3 - wave};
    int i[2];
    float Gi[2];
    SplitFrag q[2][NK];
    u32x4 sf[2][NK][2];
    auto request = [&](int v) {
        const u32x4 *src = w.s + ((ch * w.nv + min(v, w.nv - 1)) * NK * 2) * 64 + lane;
#pragma unroll
        for (int kk = 0; kk < NK; ++kk) sf[v & 1][kk][0] = src[kk * 128], sf[v & 1][kk][1] = src[kk * 128 + 64];
    };
    request(0);
#pragma unroll
    for (int t = 0; t < 2; ++t) {
        i[t] = tile[t] * 16 + r16;
        Gi[t] = sG[i[t]];
#pragma unroll
        for (int kk = 0; kk < NK; ++kk) q[t][kk] = load(Q, i[t], kk);
    }
    f32x4 o[NV][2];
    const float ei[2] = {expf(Gi[0]), expf(Gi[1])};
#pragma unroll
    for (int v = 0; v < NV; ++v) {
        if (v + 1 < NV) request(v + 1);
        __builtin_amdgcn_sched_barrier(0);
#pragma unroll
        for (int t = 0; t < 2; ++t) o[v][t] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int kk = 0; kk < NK; ++kk) {
            const bf16x8 hi = __builtin_bit_cast(bf16x8, sf[v & 1][kk][0]), lo = __builtin_bit_cast(bf16x8, sf[v & 1][kk][1]);
#pragma unroll
            for (int t = 0; t < 2; ++t) o[v][t] = mfma_bf16(hi, q[t][kk].hi, o[v][t]);
#pragma unroll
            for (int t = 0; t < 2; ++t) o[v][t] = mfma_bf16(hi, q[t][kk].lo, o[v][t]);
#pragma unroll
            for (int t = 0; t < 2; ++t) o[v][t] = mfma_bf16(lo, q[t][kk].hi, o[v][t]);
        }
#pragma unroll
        for (int t = 0; t < 2; ++t) o[v][t] *= ei[t];
        __builtin_amdgcn_sched_barrier(0);
    }
    // tokens 32 k2 .. 32 k2 + 31: both tiles look at the first half, the later one at the second
#pragma unroll
    for (int k2 = 0; k2 < 2; ++k2) {
        SplitFrag b[2];
        f32x4 s[2][2];
#pragma unroll
        for (int j = 0; j < 2; ++j) {
#pragma unroll
            for (int t = k2; t < 2; ++t) s[t][j] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int kk = 0; kk < NK; ++kk) {
                const SplitFrag k = load(K, (k2 * 2 + j) * 16 + r16, kk);
#pragma unroll
                for (int t = k2; t < 2; ++t) s[t][j] = mfma_split(k, q[t][kk], s[t][j]);
            }
#pragma unroll
            for (int t = k2; t < 2; ++t)
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    const int at = (k2 * 2 + j) * 16 + g * 4 + e;
                    s[t][j][e] = at <= i[t] ? s[t][j][e] * expf(Gi[t] - sG[at]) : 0.f;
                }
        }
#pragma unroll
        for (int t = k2; t < 2; ++t) b[t] = split8(s[t][0], s[t][1]);
        u32x4 uf[2][2];
        auto request_u = [&](int v) {
            const u32x4 *src = w.u + (((ch * w.nv + min(v, w.nv - 1)) * 2 + k2) * 2) * 64 + lane;
            uf[v & 1][0] = src[0], uf[v & 1][1] = src[64];
        };
        request_u(0);
#pragma unroll
        for (int v = 0; v < NV; ++v) {
            if (v + 1 < NV) request_u(v + 1);
            __builtin_amdgcn_sched_barrier(0);
            const bf16x8 hi = __builtin_bit_cast(bf16x8, uf[v & 1][0]), lo = __builtin_bit_cast(bf16x8, uf[v & 1][1]);
#pragma unroll
            for (int t = k2; t < 2; ++t) {
                o[v][t] = mfma_bf16(hi, b[t].hi, o[v][t]);
                o[v][t] = mfma_bf16(hi, b[t].lo, o[v][t]);
                o[v][t] = mfma_bf16(lo, b[t].hi, o[v][t]);
            }
            __builtin_amdgcn_sched_barrier(0);
        }
    }
#pragma unroll
    for (int t = 0; t < 2; ++t) {
        float ss = 0.f;
#pragma unroll
        for (int v = 0; v < NV; ++v)
            if (v < w.nv) ss += (o[v][t].x * o[v][t].x + o[v][t].y * o[v][t].y) + (o[v][t].z * o[v][t].z + o[v][t].w * o[v][t].w);
        const float inv = 1.0f / sqrtf(rows_sum(ss) / (float)p.vdim + p.eps);
        if (i[t] >= len) continue;
        const uint16_t *gate = rows + (size_t)(t0 + i[t]) * ld + C + (size_t)h * vdimp + g * 4;
        uint16_t *dst = out + (size_t)(t0 + i[t]) * ldo + (size_t)h * vdimp + g * 4;
#pragma unroll
        for (int v = 0; v < NV; ++v)
            if (v < w.nv) {
                const u32x2 gb = *reinterpret_cast<const u32x2 *>(gate + v * 16);
                const f32x4 nw = *reinterpret_cast<const f32x4 *>(p.norm + v * 16 + g * 4);
                const f32x4 ga = f32x4{bf2f(gb.x & 0xffffu), bf2f(gb.x >> 16), bf2f(gb.y & 0xffffu), bf2f(gb.y >> 16)};
                f32x4 r = o[v][t] * inv * nw;
#pragma unroll
                for (int e = 0; e < 4; ++e) r[e] *= ga[e] * __builtin_amdgcn_rcpf(1.0f + __expf(-ga[e]));
                *reinterpret_cast<bf16x4 *>(dst + v * 16) = bf16x4{(__bf16)r.x, (__bf16)r.y, (__bf16)r.z, (__bf16)r.w};
            }
    }
}

// bytes of one chunk and head: w, k (same size), ut, s, u, g
static size_t chunk_bytes(size_t nk, size_t nv) { return 2 * (4 * nk * 2048) + nv * 4096 + nv * nk * 2048 + nv * 4096 + 256; }

static size_t segment_chunks(size_t heads) { return std::max((size_t)kDeltaUnits / heads, (size_t)4); }

size_t delta_workspace_bytes(size_t n, size_t heads, size_t dimp, size_t vdimp) {
    return std::min((n + kDeltaChunk - 1) / kDeltaChunk, segment_chunks(heads)) * heads * chunk_bytes(dimp / 32, vdimp / 16);
}

template <int NK>
static hipError_t out_nv(const Delta &d, const float *qk, const uint16_t *rows, size_t ld, int n, const DeltaWs &w, uint16_t *out, size_t ldo, hipStream_t s) {
    auto fn = w.nv <= 4 ? k_delta_out<NK, 4> : w.nv <= 8 ? k_delta_out<NK, 8> : k_delta_out<NK, 16>;
    hipLaunchKernelGGL(fn, dim3(w.nc, d.heads), dim3(128), 0, s, d, qk, rows, ld, n, w, out, ldo);
    return hipGetLastError();
}

hipError_t launch_delta_chunked(const Delta &d, const float *qk, const uint16_t *v, const float *gates, const uint16_t *rows, size_t ld, int n,
                                uint16_t *out, size_t ldo, void *workspace, hipStream_t s) {
    if (!delta_chunked_supported((int)d.dimp, (int)d.vdimp)) return hipErrorInvalidValue;
    const size_t lds = (64 * (d.dimp + 4) + 2 * 64 * kTriStride) * sizeof(float);
    if (lds > 65536) {
        const hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void *>(k_delta_chunk), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
        if (e != hipSuccess) return e;
    }
    const int segment = (int)segment_chunks(d.heads) * kDeltaChunk;
    for (int t0 = 0; t0 < n; t0 += segment) {
        const int m = min(segment, n - t0);
        DeltaWs w;
        w.nc = (m + kDeltaChunk - 1) / kDeltaChunk, w.nk = (int)d.dimp / 32, w.nv = (int)d.vdimp / 16;
        const size_t ch = (size_t)w.nc * d.heads, nk = w.nk, nv = w.nv;
        w.w = (u32x4 *)workspace;
        w.k = w.w + ch * 4 * nk * 128;
        w.ut = (f32x4 *)(w.k + ch * 4 * nk * 128);
        w.s = (u32x4 *)(w.ut + ch * nv * 256);
        w.u = w.s + ch * nv * nk * 128;
        w.g = (float *)(w.u + ch * nv * 256);
        const float *q = qk + (size_t)t0 * 2 * d.kv_heads * d.dimp, *gt = gates + (size_t)t0 * 2 * d.heads;
        const uint16_t *vv = v + (size_t)t0 * d.heads * d.vdimp, *rr = rows + (size_t)t0 * ld;
        uint16_t *oo = out + (size_t)t0 * ldo;
        hipLaunchKernelGGL(k_delta_chunk, dim3(w.nc, d.heads), dim3(256), lds, s, d, q, vv, gt, m, w);
        const dim3 grid(8 * ((d.heads + 7) / 8) * w.nv);
        auto scan = nk == 1 ? k_delta_scan<1> : nk == 2 ? k_delta_scan<2> : nk == 3 ? k_delta_scan<3> : k_delta_scan<4>;
        hipLaunchKernelGGL(scan, grid, dim3(256), 0, s, d, w);
        const hipError_t e = nk == 1 ? out_nv<1>(d, q, rr, ld, m, w, oo, ldo, s) : nk == 2 ? out_nv<2>(d, q, rr, ld, m, w, oo, ldo, s)
                           : nk == 3 ? out_nv<3>(d, q, rr, ld, m, w, oo, ldo, s) : out_nv<4>(d, q, rr, ld, m, w, oo, ldo, s);
        if (e != hipSuccess) return e;
    }
    return hipGetLastError();
}

}  // namespace bitnet_hip
