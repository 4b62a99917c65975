// kernels_gqa.hip -- causal attention whose query heads share keys and values in groups, with one softmax map per head or two (gfx950).
// Optionally rotated queries and keys, chunks of positions that do not see each other, a window, a penalty that grows with the distance, a sink in the
// softmax's denominator, keys that are the values too, short convolutions ahead of it all, and a gate per head or column on the output.
//
// Two maps (differential attention) weigh the same values; a head's output is a1 - lambda a2, divided by its root mean square over the value
// columns.  Caches: keys [kv head][map][capacity][dimp], values transposed [kv head][vdimp][capacity].
//   k_gqa_rows     rows of projections: convolution, query and key norms, the query's factor at its position, keys and values into the caches
//   k_gqa_prefill  a prompt's portion: flash attention on S^T = K Q^T and O^T = V^T P^T, both maps of a query tile in one wave
//   k_gqa_step     the decode step: norms and append in the same launch, 32 keys per wave and step on the matrix cores
//   k_gqa_any      any size, f32 or bf16 cache, one wave per key
//   k_gqa_merge    records of the decode forms -> output
// Scores, maxima, sums and weights are f32; a weight (and the decode step's query) enters the matrix cores as a (high, low) pair of bf16 values.
// Scores are kept in base 2: the score times log2(e).
#include "dense.hpp"

namespace bitnet_hip {

constexpr float kLog2e = 1.44269504088896f;

// the first key a query at this position sees
__device__ __forceinline__ int gqa_first(const Gqa &p, int pos) {
    const int first = p.chunk ? pos - (int)((unsigned)pos % (unsigned)p.chunk) : 0;
    return p.window ? max(first, pos - (int)p.window + 1) : first;
}

// The records of a query at `pos`: tiles of keys from `base` (the tile that holds its first key) on, `per` tiles each.
struct GqaRange {
    int first, base, per, used;
};
__device__ __forceinline__ GqaRange gqa_range(const Gqa &p, int pos) {
    GqaRange r;
    r.first = gqa_first(p, pos);
    r.base = r.first & ~(kGqaTile - 1);
    const int tiles = (pos + 1 - r.base + kGqaTile - 1) / kGqaTile;
    r.per = (tiles + kGqaSplits - 1) / kGqaSplits;
    r.used = (tiles + r.per - 1) / r.per;
    return r;
}
// records a launch has to provide for
static int gqa_records(const Gqa &g) {
    size_t keys = g.capacity;
    if (g.chunk && g.chunk + kGqaTile < keys) keys = g.chunk + kGqaTile;  // (a chunk may start inside a tile)
    if (g.window && g.window + kGqaTile < keys) keys = g.window + kGqaTile;
    return (int)min((size_t)kGqaSplits, (keys + kGqaTile - 1) / kGqaTile);
}

// element i of a head at a position, v being its own and the lane's neighbour holding the other element of the pair; cs, sn: the tables' row
__device__ __forceinline__ float turn_neighbours(float v, int i, const float *cs, const float *sn, int dims) {
    const float o = dpp<0xb1>(v);  // quad_perm [1,0,3,2]
    if (i >= dims) return v;
    const float c = cs[i >> 1], s = sn[i >> 1];
    return (i & 1) ? v * c + o * s : v * c - o * s;
}
// what a head's gate (or that of a column of it) is the sigmoid of
__device__ __forceinline__ float gate_logit(const Gqa &p, int row, int h, int column) {
    const size_t i = (size_t)row * p.ldgate + (p.gate_columns ? (size_t)h * p.vdimp + column : (size_t)h);
    return p.gate_f32 ? ((const float *)p.gate)[i] : bf2f(((const uint16_t *)p.gate)[i]);
}
// a head's distance penalty: what is taken off the natural score is weight * log2(1 + rate * distance)
struct FarPenalty {
    float weight, rate;
};
__device__ __forceinline__ FarPenalty far_penalty(const Gqa &p, int h) {
    FarPenalty f{0.f, 0.f};
    if (p.far_weight) f.weight = p.far_weight[h] * 0.69314718055994531f, f.rate = p.far_rate[h];
    return f;
}
__device__ __forceinline__ float nearer(float score, const FarPenalty &f, int distance) { return fmaf(-f.weight, __log2f(fmaf(f.rate, (float)distance, 1.0f)), score); }
// columns of a row of projections that a convolution covers
__host__ __device__ __forceinline__ int gqa_channels(const Gqa &p) {
    if (p.queries_only) return (int)(p.heads * p.maps * p.dimp);
    return (int)((p.heads + p.kv_heads) * p.maps * p.dimp + (p.values_are_keys ? 0 : p.kv_heads * p.vdimp));
}
// column c of the row of projections t (negative: an earlier portion's; zero ahead of the sequence)
template <class TR>
__device__ __forceinline__ float raw_value(const Gqa &p, const TR *rows, size_t ld, int pos0, int t, int c, int channels) {
    if (t >= 0) return ld_act(rows + (size_t)t * ld, c);
    const int at = pos0 + t;
    return at >= 0 ? p.ring[(size_t)(at % (int)p.taps) * channels + c] : 0.f;
}

size_t gqa_scratch_floats(size_t heads, size_t maps, size_t vdimp, size_t nq) { return nq * heads * maps * kGqaSplits * (kGqaRecHead + vdimp); }
bool gqa_supported(int dimp, int vdimp) { return dimp <= 256 && vdimp <= 256; }

// ---- rows of projections ----------------------------------------------------------------------------------------------
// blockIdx.y: query heads x maps, key heads x maps (sixteen tokens per workgroup, four per wave), then value heads in groups of 32 columns (64
// tokens, every fourth workgroup).
constexpr int kRowTokens = 16, kRowCols = 32;

// Four tokens of a query or key head of up to 128 NJ columns: a lane holds neighbouring elements, so that a pair turns within it.  TAPS: those of the convolution
// (0: none, -1: any number).
template <class TR, class TC, int NJ, int TAPS>
__device__ __forceinline__ void head_rows(const Gqa &p, const TR *rows, size_t ld, int pos0, int t0, int n, int y, bool key, TC *cache, TR *queries, size_t ldq) {
    constexpr int U = kRowTokens / 4;
    constexpr bool CONV = TAPS != 0;
    const int lane = threadIdx.x & 63, dim = (int)p.dim, dimp = (int)p.dimp, turned = (int)p.rot_dims, half = turned >> 1;
    const float *w = key ? p.k_weight : p.q_weight;
    float v[U][NJ][2], cs[U][NJ], sn[U][NJ], factor[U];
#pragma unroll
    for (int u = 0; u < U; ++u) {
        const int t = min(t0 + u, n - 1);
        const TR *row = rows + (size_t)t * ld + (size_t)y * dimp;
        factor[u] = key ? 1.0f : p.q_factor[pos0 + t];
#pragma unroll
        for (int j = 0; j < NJ; ++j) {
            const int i = min(2 * lane + 128 * j, dimp - 2);
            if (CONV)
                v[u][j][0] = v[u][j][1] = 0.f;
            else
                v[u][j][0] = ld_act(row, i), v[u][j][1] = ld_act(row, i + 1);
            cs[u][j] = 1.0f, sn[u][j] = 0.f;
            if (turned && 2 * lane + 128 * j < turned) {
                const size_t at = (size_t)(pos0 + t) * half + lane + 64 * j;
                cs[u][j] = p.rope_cos[at], sn[u][j] = p.rope_sin[at];
            }
        }
    }
    if (TAPS > 0) {  // the tokens and those ahead of them once, in registers
        constexpr int T = TAPS > 0 ? TAPS : 1;
        const int channels = gqa_channels(p);
#pragma unroll
        for (int j = 0; j < NJ; ++j) {
            const int c = y * dimp + min(2 * lane + 128 * j, dimp - 2);
            float f[T][2], raw[U + T - 1][2];
#pragma unroll
            for (int k = 0; k < T; ++k) f[k][0] = p.conv[(size_t)k * channels + c], f[k][1] = p.conv[(size_t)k * channels + c + 1];
            if (t0 >= T - 1) {
#pragma unroll
                for (int k = 0; k < U + T - 1; ++k) {
                    const TR *row = rows + (size_t)min(t0 - (T - 1) + k, n - 1) * ld;
                    raw[k][0] = ld_act(row, c), raw[k][1] = ld_act(row, c + 1);
                }
            } else {
#pragma unroll
                for (int k = 0; k < U + T - 1; ++k) {
                    const int t = min(t0 - (T - 1) + k, n - 1);
                    raw[k][0] = raw_value(p, rows, ld, pos0, t, c, channels), raw[k][1] = raw_value(p, rows, ld, pos0, t, c + 1, channels);
                }
            }
#pragma unroll
            for (int u = 0; u < U; ++u)
#pragma unroll
                for (int k = 0; k < T; ++k) v[u][j][0] += f[k][0] * raw[u + k][0], v[u][j][1] += f[k][1] * raw[u + k][1];
        }
    } else if (CONV) {
        const int taps = (int)p.taps, channels = gqa_channels(p);
        for (int k = 0; k < taps; ++k)
#pragma unroll
            for (int j = 0; j < NJ; ++j) {
                const int c = y * dimp + min(2 * lane + 128 * j, dimp - 2);
                const float f0 = p.conv[(size_t)k * channels + c], f1 = p.conv[(size_t)k * channels + c + 1];
#pragma unroll
                for (int u = 0; u < U; ++u) {
                    const int t = min(t0 + u, n - 1) - (taps - 1) + k;
                    v[u][j][0] += f0 * raw_value(p, rows, ld, pos0, t, c, channels), v[u][j][1] += f1 * raw_value(p, rows, ld, pos0, t, c + 1, channels);
                }
            }
    }
    float wv[NJ][2];
#pragma unroll
    for (int j = 0; j < NJ; ++j)
#pragma unroll
        for (int e = 0; e < 2; ++e) wv[j][e] = w && 2 * lane + 128 * j + e < dim ? w[2 * lane + 128 * j + e] : 1.0f;  // (padding columns hold zeros)
#pragma unroll
    for (int u = 0; u < U; ++u) {
        if (w || p.unit_norm) {
            float ss = 0.f;
#pragma unroll
            for (int j = 0; j < NJ; ++j) ss += 2 * lane + 128 * j < dimp ? v[u][j][0] * v[u][j][0] + v[u][j][1] * v[u][j][1] : 0.f;
            factor[u] *= 1.0f / sqrtf(wave_sum(ss) / (float)dim + p.eps);
        }
        if (t0 + u >= n) continue;
        TR *row = queries + (size_t)(t0 + u) * ldq + (size_t)y * dimp;
#pragma unroll
        for (int j = 0; j < NJ; ++j) {
            const int i = 2 * lane + 128 * j;
            if (i >= dimp) continue;
            const float a = v[u][j][0] * factor[u] * wv[j][0], b = v[u][j][1] * factor[u] * wv[j][1];
            const float x = a * cs[u][j] - b * sn[u][j], z = b * cs[u][j] + a * sn[u][j];
            if (key) {
                TC *dst = cache + (size_t)(pos0 + t0 + u) * dimp;
                st_act(dst, i, x), st_act(dst, i + 1, z);
            } else {
                st_act(row, i, x), st_act(row, i + 1, z);
            }
        }
    }
}

// TAPS (as head_rows): every column passes a convolution over time first, and the queries go to a place of their own
template <class TR, class TC, int NJ, int TAPS>
__global__ __launch_bounds__(256) void k_gqa_rows(Gqa p, const TR *rows, size_t ld, const int *pos_ptr, int n, TR *queries, size_t ldq) {
    constexpr int STRIDE = sizeof(TR) == 4 ? kRowCols + 1 : kRowCols + 2;
    constexpr bool CONV = TAPS != 0;
    __shared__ __attribute__((aligned(16))) TR tile[(64 + (TAPS < 0 ? kMaxTaps - 1 : TAPS > 0 ? TAPS - 1 : 0)) * STRIDE];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, pos0 = *pos_ptr;
    const int nq = (int)(p.heads * p.maps), nk = (int)(p.kv_heads * p.maps), dim = (int)p.dim, dimp = (int)p.dimp, vdimp = (int)p.vdimp;
    int y = blockIdx.y;
    if (y < nq + nk) {
        const bool key = y >= nq;
        const float *w = key ? p.k_weight : p.q_weight;
        const int turned = (int)p.rot_dims, half = turned >> 1, t0 = blockIdx.x * kRowTokens + wave * (kRowTokens / 4);
        TC *cache = key ? (TC *)p.kcache + (size_t)(y - nq) * p.capacity * dimp : nullptr;
        if (t0 >= n) return;
        if (dimp <= 128 * NJ) {
            head_rows<TR, TC, NJ, TAPS>(p, rows, ld, pos0, t0, n, y, key, cache, queries, ldq);
            return;
        }
        const int channels = gqa_channels(p), taps = (int)p.taps;
        for (int t = t0; t < min(t0 + kRowTokens / 4, n); ++t) {
            TR *row = queries + (size_t)t * ldq + (size_t)y * dimp;
            auto value = [&](int i) {
                if (!CONV) return ld_act(rows + (size_t)t * ld + (size_t)y * dimp, i);
                float v = 0.f;
                for (int k = 0; k < taps; ++k) v += p.conv[(size_t)k * channels + y * dimp + i] * raw_value(p, rows, ld, pos0, t - (taps - 1) + k, y * dimp + i, channels);
                return v;
            };
            float ss = 0.f;
            if (w || p.unit_norm)
                for (int i = lane; i < dimp; i += 64) {
                    const float v = value(i);
                    ss += v * v;
                }
            const float norm = w || p.unit_norm ? 1.0f / sqrtf(wave_sum(ss) / (float)dim + p.eps) : 1.0f;
            const float factor = key ? norm : norm * p.q_factor[pos0 + t];
            const float *cs = p.rope_cos + (size_t)(pos0 + t) * half, *sn = p.rope_sin + (size_t)(pos0 + t) * half;
            for (int i = lane; i < dimp; i += 64) {
                float v = value(i) * factor * (w && i < dim ? w[i] : 1.0f);
                if (turned) v = turn_neighbours(v, i, cs, sn, turned);
                if (key)
                    st_act(cache + (size_t)(pos0 + t) * dimp, i, v);
                else
                    st_act(row, i, v);
            }
        }
        return;
    }
    if (blockIdx.x % (64 / kRowTokens)) return;
    y -= nq + nk;
    const int t0 = blockIdx.x * kRowTokens, groups = vdimp / kRowCols, head = y / groups, c0 = (y - head * groups) * kRowCols, count = min(64, n - t0);
    const int column = (p.values_are_keys ? nq : nq + nk) * dimp + head * vdimp + c0;
    const TR *src = rows + column;
    constexpr int V = 16 / sizeof(TR), PER = kRowCols / V;
    const int taps = TAPS > 0 ? TAPS : CONV ? (int)p.taps : 1, channels = gqa_channels(p);
    if (CONV) {  // the tokens ahead of the first one in the tile's last rows
        for (int i = tid; i < (taps - 1) * kRowCols; i += 256) {
            const int k = i / kRowCols, c = i % kRowCols;
            st_act(tile, (64 + k) * STRIDE + c, raw_value(p, rows, ld, pos0, t0 - (taps - 1) + k, column + c, channels));
        }
    }
#pragma unroll
    for (int j = 0; j < 64 * PER / 256; ++j) {
        const int i = tid + 256 * j, t = i / PER, c = i % PER * V;
        if (t < count) {
            const u32x4 x = *reinterpret_cast<const u32x4 *>(src + (size_t)(t0 + t) * ld + c);
            uint32_t *dst = reinterpret_cast<uint32_t *>(tile + t * STRIDE + c);
            dst[0] = x.x, dst[1] = x.y, dst[2] = x.z, dst[3] = x.w;
        }
    }
    __syncthreads();
    TC *cache = (TC *)p.vcache + ((size_t)head * vdimp + c0) * p.capacity + pos0 + t0;
    if (lane < count)
#pragma unroll
        for (int j = 0; j < kRowCols / 4; ++j) {
            const int v = wave * (kRowCols / 4) + j;
            float x;
            if (CONV) {
                x = 0.f;
#pragma unroll TAPS > 0 ? TAPS : 1
                for (int k = 0; k < taps; ++k) {
                    const int t = lane - (taps - 1) + k;
                    x += p.conv[(size_t)k * channels + column + v] * ld_act(tile, (t >= 0 ? t : 64 + taps - 1 + t) * STRIDE + v);
                }
            } else {
                x = ld_act(tile, lane * STRIDE + v);
            }
            st_act(cache + (size_t)v * p.capacity, lane, x);
        }
}

template <class TR, class TC>
static hipError_t rows_go(const Gqa &g, const void *rows, size_t ld, const int *pos, int n, void *q, size_t ldq, hipStream_t s) {
    const int keys = g.queries_only ? 0 : (int)(g.kv_heads * g.maps + g.kv_heads * (g.vdimp / kRowCols));
    const dim3 grid((n + kRowTokens - 1) / kRowTokens, (int)(g.heads * g.maps) + keys);
    auto pick = [&](auto narrow, auto wide) { return g.dimp <= 128 ? narrow : wide; };
    auto fn = g.taps == 0   ? pick(k_gqa_rows<TR, TC, 1, 0>, k_gqa_rows<TR, TC, 2, 0>)
              : g.taps == 2 ? pick(k_gqa_rows<TR, TC, 1, 2>, k_gqa_rows<TR, TC, 2, 2>)
              : g.taps == 3 ? pick(k_gqa_rows<TR, TC, 1, 3>, k_gqa_rows<TR, TC, 2, 3>)
              : g.taps == 4 ? pick(k_gqa_rows<TR, TC, 1, 4>, k_gqa_rows<TR, TC, 2, 4>)
                            : pick(k_gqa_rows<TR, TC, 1, -1>, k_gqa_rows<TR, TC, 2, -1>);
    hipLaunchKernelGGL(fn, grid, dim3(256), 0, s, g, (const TR *)rows, ld, pos, n, (TR *)q, ldq);
    return hipGetLastError();
}

hipError_t launch_gqa_rows(const Gqa &g, void *rows, size_t ld, int rows_f32, int cache_f32, const int *pos, int n, void *q, size_t ldq, hipStream_t s) {
    if (rows_f32) return cache_f32 ? rows_go<float, float>(g, rows, ld, pos, n, q, ldq, s) : rows_go<float, uint16_t>(g, rows, ld, pos, n, q, ldq, s);
    return cache_f32 ? hipErrorInvalidValue : rows_go<uint16_t, uint16_t>(g, rows, ld, pos, n, q, ldq, s);
}

// ---- any size ---------------------------------------------------------------------------------------------------------
// One workgroup per (record, head and map, query); a wave takes every fourth key, its lanes the columns.
template <class TQ, class TC, int ND, int NV>
__global__ __launch_bounds__(256) void k_gqa_any(Gqa p, const TQ *q, size_t ldq, const int *pos_ptr, int q0, float *scratch) {
    extern __shared__ __attribute__((aligned(16))) float vec[];  // [4][vdimp]
    __shared__ float sm[4], sl[4];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, hm = blockIdx.y, qi = blockIdx.z;
    const int maps = (int)p.maps, h = hm / maps, map = hm - h * maps, kv = h / (int)(p.heads / p.kv_heads), dimp = (int)p.dimp, vdimp = (int)p.vdimp;
    const int pos = *pos_ptr + q0 + qi;
    const GqaRange range = gqa_range(p, pos);
    if ((int)blockIdx.x >= range.used) return;
    const int start = range.base + blockIdx.x * range.per * kGqaTile, k0 = max(start, range.first), k1 = min(start + range.per * kGqaTile, pos + 1);
    const TQ *qr = q + (size_t)qi * ldq + (size_t)hm * dimp;
    const TC *K = (const TC *)p.kcache + (size_t)(kv * maps + map) * p.capacity * dimp, *V = (const TC *)p.vcache + (size_t)kv * vdimp * p.capacity;
    float qv[ND], acc[NV];
#pragma unroll
    for (int j = 0; j < ND; ++j) qv[j] = lane + 64 * j < dimp ? ld_act(qr, lane + 64 * j) : 0.f;
#pragma unroll
    for (int j = 0; j < NV; ++j) acc[j] = 0.f;
    const FarPenalty far = far_penalty(p, h);
    float m = -INFINITY, l = 0.f;
    for (int key = k0 + wave; key < k1; key += 4) {
        float s = 0.f;
#pragma unroll
        for (int j = 0; j < ND; ++j)
            if (lane + 64 * j < dimp) s += qv[j] * ld_act(K + (size_t)key * dimp, lane + 64 * j);
        s = nearer(wave_sum(s), far, pos - key) * kLog2e;
        const float mn = fmaxf(m, s), al = exp2f(m - mn), w = exp2f(s - mn);
        l = l * al + w;
        m = mn;
#pragma unroll
        for (int j = 0; j < NV; ++j)
            if (lane + 64 * j < vdimp) acc[j] = acc[j] * al + w * ld_act(V + (size_t)(lane + 64 * j) * p.capacity, key);
    }
    if (lane == 0) sm[wave] = m, sl[wave] = l;
#pragma unroll
    for (int j = 0; j < NV; ++j)
        if (lane + 64 * j < vdimp) vec[wave * vdimp + lane + 64 * j] = acc[j];
    __syncthreads();
    const float M = fmaxf(fmaxf(sm[0], sm[1]), fmaxf(sm[2], sm[3]));
    float w[4], L = 0.f;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
        w[i] = sm[i] == -INFINITY ? 0.f : exp2f(sm[i] - M);
        L += w[i] * sl[i];
    }
    float *rec = scratch + (((size_t)qi * p.heads * maps + hm) * kGqaSplits + blockIdx.x) * (kGqaRecHead + vdimp);
    for (int i = tid; i < vdimp; i += 256)
        rec[kGqaRecHead + i] = (w[0] * vec[i] + w[1] * vec[vdimp + i]) + (w[2] * vec[2 * vdimp + i] + w[3] * vec[3 * vdimp + i]);
    if (tid == 0) rec[0] = M, rec[1] = L;
}

template <class TQ, class TC>
static hipError_t any_go(const Gqa &g, const void *q, size_t ldq, const int *pos, int q0, int nq, float *scratch, hipStream_t s) {
    const int splits = gqa_records(g);
    const size_t lds = 4 * g.vdimp * sizeof(float);
    if (g.dimp > 1024 || g.vdimp > 1024) return hipErrorInvalidValue;
    auto fn = g.dimp <= 64 && g.vdimp <= 64 ? k_gqa_any<TQ, TC, 1, 1> : g.dimp <= 256 && g.vdimp <= 256 ? k_gqa_any<TQ, TC, 4, 4> : k_gqa_any<TQ, TC, 16, 16>;
    hipLaunchKernelGGL(fn, dim3(splits, g.heads * g.maps, nq), dim3(256), lds, s, g, (const TQ *)q, ldq, pos, q0, scratch);
    return hipGetLastError();
}

hipError_t launch_gqa_any(const Gqa &g, const void *q, size_t ldq, int q_f32, int cache_f32, const int *pos, int q0, int nq, float *scratch, hipStream_t s) {
    if (q_f32) return cache_f32 ? any_go<float, float>(g, q, ldq, pos, q0, nq, scratch, s) : any_go<float, uint16_t>(g, q, ldq, pos, q0, nq, scratch, s);
    return cache_f32 ? hipErrorInvalidValue : any_go<uint16_t, uint16_t>(g, q, ldq, pos, q0, nq, scratch, s);
}

// ---- decode step, matrix cores ----------------------------------------------------------------------------------------
// One workgroup per (record, kv head and 16 of its query heads), four waves; a wave takes every fourth block of 32 keys by itself, with maximum,
// sum and output of its own, and the four meet at the end.  S^T = K Q^T: row 4 g + e of score tile t is key 8 g + 4 t + e of the block, so that a
// lane's weights of both tiles are the eight consecutive keys 8 g .. 8 g + 7 which it needs as an operand of O^T = V^T P^T.
template <int NK, int NV, int MAPS>
__global__ __launch_bounds__(256, NV > 8 || NK * MAPS >= 8 ? 1 : 2) void k_gqa_step(Gqa p, GqaStep a) {
    extern __shared__ __attribute__((aligned(16))) float area[];  // queries [maps][16][NK * 32]; then the waves' outputs
    __shared__ float sm[4][MAPS][16], sl[4][MAPS][16];
    __shared__ __attribute__((aligned(16))) uint16_t newk[MAPS][NK * 32], newv[NV * 16];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, r16 = lane & 15, g = lane >> 4;
    const int group = (int)(p.heads / p.kv_heads), ht = (group + 15) / 16, kv = blockIdx.y / ht, h0 = kv * group + (blockIdx.y - kv * ht) * 16;
    const int nh = min(16, (kv + 1) * group - h0), dim = (int)p.dim, dimp = (int)p.dimp, vdimp = (int)p.vdimp;
    constexpr int QS = NK * 32 + 4;
    const int pos = *a.pos, n_keys = pos + 1;
    const GqaRange range = gqa_range(p, pos);
    if ((int)blockIdx.x >= range.used) return;
    const int k0 = range.base + blockIdx.x * range.per * kGqaTile, k1 = min(k0 + range.per * kGqaTile, n_keys);
    uint16_t *K = (uint16_t *)p.kcache + (size_t)kv * MAPS * p.capacity * dimp, *V = (uint16_t *)p.vcache + (size_t)kv * vdimp * p.capacity;
    const float *kraw = a.row + (p.heads * MAPS + (size_t)kv * MAPS) * dimp,
                *vraw = p.values_are_keys ? kraw : a.row + (p.heads + p.kv_heads) * MAPS * dimp + (size_t)kv * vdimp;
    const int turned = (int)p.rot_dims;
    const float *cs = p.rope_cos + (size_t)pos * (turned >> 1), *sn = p.rope_sin + (size_t)pos * (turned >> 1);
    u32x4 kf[2][MAPS][NK], vf[NV];
    auto fetch = [&](int kb) {  // (blocks lie below the capacity, a multiple of 128)
#pragma unroll
        for (int t = 0; t < 2; ++t)
#pragma unroll
            for (int j = 0; j < MAPS; ++j)
#pragma unroll
                for (int kk = 0; kk < NK; ++kk)
                    kf[t][j][kk] = *reinterpret_cast<const u32x4 *>(K + ((size_t)j * p.capacity + kb + (r16 >> 2) * 8 + t * 4 + (r16 & 3)) * dimp + min(kk * 32, dimp - 32) + g * 8);
#pragma unroll
        for (int v = 0; v < NV; ++v) vf[v] = *reinterpret_cast<const u32x4 *>(V + (size_t)min(v * 16 + r16, vdimp - 1) * p.capacity + kb + g * 8);
    };
    constexpr bool kAhead = NK <= 4;  // the first block is requested ahead of the norms (registers allow it)
    const bool owner = k1 == n_keys && !p.queries_only;
    if (kAhead) fetch(k0 + wave * 32);
    if (owner) {  // the record that holds the new position appends it (and puts it into its own fragments below)
        if (wave < MAPS) {
            float v[NK], ss = 0.f;
#pragma unroll
            for (int j = 0; j < (NK + 1) / 2; ++j) {
                v[j] = lane + 64 * j < dimp ? kraw[wave * dimp + lane + 64 * j] : 0.f;
                ss += v[j] * v[j];
            }
            const float norm = p.k_weight || p.unit_norm ? 1.0f / sqrtf(wave_sum(ss) / (float)dim + p.eps) : 1.0f;
#pragma unroll
            for (int j = 0; j < (NK + 1) / 2; ++j) {
                const int i = lane + 64 * j;
                float k = v[j] * norm * (p.k_weight && i < dim ? p.k_weight[i] : 1.0f);
                if (turned) k = turn_neighbours(k, i, cs, sn, turned);
                if (i < dimp) {
                    const uint16_t b = f2bf(k);
                    K[((size_t)wave * p.capacity + pos) * dimp + i] = b;
                    newk[wave][i] = b;
                }
            }
        }
        for (int i = tid; i < vdimp; i += 256) {
            const uint16_t b = f2bf(vraw[i]);
            V[(size_t)i * p.capacity + pos] = b;
            newv[i] = b;
        }
    }
    {
        const float factor = p.q_factor[pos];
        for (int r = wave; r < MAPS * 16; r += 4) {
            const int map = r >> 4, hh = r & 15;
            if (hh >= nh) {
                for (int i = lane; i < NK * 32; i += 64) area[r * QS + i] = 0.f;
                continue;
            }
            const float *q = a.row + ((size_t)(h0 + hh) * MAPS + map) * dimp;
            float v[NK], ss = 0.f;
#pragma unroll
            for (int j = 0; j < (NK + 1) / 2; ++j) {
                v[j] = lane + 64 * j < dimp ? q[lane + 64 * j] : 0.f;
                ss += v[j] * v[j];
            }
            const float norm = (p.q_weight || p.unit_norm ? 1.0f / sqrtf(wave_sum(ss) / (float)dim + p.eps) : 1.0f) * factor;
#pragma unroll
            for (int j = 0; j < (NK + 1) / 2; ++j) {
                const int i = lane + 64 * j;
                float t = v[j] * norm * (p.q_weight && i < dim ? p.q_weight[i] : 1.0f);
                if (turned) t = turn_neighbours(t, i, cs, sn, turned);
                if (i < NK * 32) area[r * QS + i] = t;
            }
        }
    }
    __syncthreads();
    SplitFrag q[MAPS][NK];
#pragma unroll
    for (int m = 0; m < MAPS; ++m)
#pragma unroll
        for (int kk = 0; kk < NK; ++kk) {
            const float *src = area + (m * 16 + r16) * QS + kk * 32 + g * 8;
            q[m][kk] = split8(*reinterpret_cast<const f32x4 *>(src), *reinterpret_cast<const f32x4 *>(src + 4));
        }
    __syncthreads();  // (the area is used again)
    const FarPenalty far = far_penalty(p, min(h0 + r16, (int)p.heads - 1));
    f32x4 o[NV][MAPS];
    float m[MAPS], l[MAPS];
#pragma unroll
    for (int j = 0; j < MAPS; ++j) {
        m[j] = -INFINITY, l[j] = 0.f;
#pragma unroll
        for (int v = 0; v < NV; ++v) o[v][j] = f32x4{0.f, 0.f, 0.f, 0.f};
    }
    for (int kb = k0 + wave * 32; kb < k1; kb += 128) {
        if (!kAhead || kb >= k0 + 128) fetch(kb);
        if (kb + 32 <= range.first) continue;  // (another chunk's keys)
        if (owner && pos - kb < 32) {  // the new position, which memory need not show yet
            const int at = pos - kb, t = (at >> 2) & 1;
            const bool mine = r16 == (at >> 3) * 4 + (at & 3);
#pragma unroll
            for (int j = 0; j < MAPS; ++j)
#pragma unroll
                for (int kk = 0; kk < NK; ++kk) {
                    const u32x4 k = *reinterpret_cast<const u32x4 *>(&newk[j][min(kk * 32, dimp - 32) + g * 8]);
                    if (mine && t == 0) kf[0][j][kk] = k;
                    if (mine && t == 1) kf[1][j][kk] = k;
                }
            if (g == at >> 3) {
                const uint32_t keep = (at & 1) ? 0xffffu : 0xffff0000u, sh = (at & 1) * 16;
#pragma unroll
                for (int v = 0; v < NV; ++v) {
                    const uint32_t n = (uint32_t)newv[min(v * 16 + r16, vdimp - 1)] << sh;
#pragma unroll
                    for (int e = 0; e < 4; ++e)
                        if (e == (at & 7) >> 1) vf[v][e] = (vf[v][e] & keep) | n;
                }
            }
        }
#pragma unroll
        for (int j = 0; j < MAPS; ++j) {
            f32x4 s[2];
#pragma unroll
            for (int t = 0; t < 2; ++t) {
                f32x4 hi = f32x4{0.f, 0.f, 0.f, 0.f}, lo = hi;
#pragma unroll
                for (int kk = 0; kk < NK; ++kk) {  // (steps past dimp: the query is zero there)
                    hi = mfma_bf16(__builtin_bit_cast(bf16x8, kf[t][j][kk]), q[j][kk].hi, hi);
                    lo = mfma_bf16(__builtin_bit_cast(bf16x8, kf[t][j][kk]), q[j][kk].lo, lo);
                }
                s[t] = hi + lo;
                if (MAPS == 1 && p.far_weight)
#pragma unroll
                    for (int e = 0; e < 4; ++e) s[t][e] = nearer(s[t][e], far, pos - (kb + g * 8 + t * 4 + e));
                s[t] *= kLog2e;
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    const int key = kb + g * 8 + t * 4 + e;
                    s[t][e] = key < k1 && key >= range.first ? s[t][e] : -INFINITY;
                }
            }
            float mx = fmaxf(fmaxf(fmaxf(s[0][0], s[0][1]), fmaxf(s[0][2], s[0][3])), fmaxf(fmaxf(s[1][0], s[1][1]), fmaxf(s[1][2], s[1][3])));
            mx = fmaxf(m[j], rows_max(mx));
            const float al = exp2f(m[j] - mx);
            m[j] = mx;
            f32x4 w[2];
#pragma unroll
            for (int t = 0; t < 2; ++t)
#pragma unroll
                for (int e = 0; e < 4; ++e) w[t][e] = exp2f(s[t][e] - mx);
            l[j] = l[j] * al + ((w[0][0] + w[0][1]) + (w[0][2] + w[0][3])) + ((w[1][0] + w[1][1]) + (w[1][2] + w[1][3]));
            const SplitFrag pf = split8(w[0], w[1]);
#pragma unroll
            for (int v = 0; v < NV; ++v) {
                o[v][j] *= al;
                o[v][j] = mfma_bf16(__builtin_bit_cast(bf16x8, vf[v]), pf.hi, o[v][j]);
                o[v][j] = mfma_bf16(__builtin_bit_cast(bf16x8, vf[v]), pf.lo, o[v][j]);
            }
        }
    }
#pragma unroll
    for (int j = 0; j < MAPS; ++j) {
        const float t = rows_sum(l[j]);
        if (g == 0) sm[wave][j][r16] = m[j], sl[wave][j][r16] = t;
    }
    __syncthreads();
#pragma unroll
    for (int j = 0; j < MAPS; ++j) {
        const float M = fmaxf(fmaxf(sm[0][j][r16], sm[1][j][r16]), fmaxf(sm[2][j][r16], sm[3][j][r16]));
        const float w = m[j] == -INFINITY ? 0.f : exp2f(m[j] - M);
        if (r16 < nh)
#pragma unroll
            for (int v = 0; v < NV; ++v)
                if (v * 16 < vdimp) *reinterpret_cast<f32x4 *>(area + ((size_t)(wave * MAPS + j) * nh + r16) * vdimp + v * 16 + g * 4) = o[v][j] * w;
    }
    __syncthreads();
    const int v4 = vdimp / 4, rows = MAPS * nh;
    for (int i = tid; i < rows * v4; i += 256) {
        const int r = i / v4, c = (i - r * v4) * 4, j = r / nh, hh = r - j * nh;
        const float *src = area + (size_t)r * vdimp + c;
        const size_t step = (size_t)rows * vdimp;
        const f32x4 sum = (*reinterpret_cast<const f32x4 *>(src) + *reinterpret_cast<const f32x4 *>(src + step)) +
                          (*reinterpret_cast<const f32x4 *>(src + 2 * step) + *reinterpret_cast<const f32x4 *>(src + 3 * step));
        float *rec = a.scratch + ((size_t)((h0 + hh) * MAPS + j) * kGqaSplits + blockIdx.x) * (kGqaRecHead + vdimp);
        *reinterpret_cast<f32x4 *>(rec + kGqaRecHead + c) = sum;
        if (c == 0) {
            const float M = fmaxf(fmaxf(sm[0][j][hh], sm[1][j][hh]), fmaxf(sm[2][j][hh], sm[3][j][hh]));
            float L = 0.f;
#pragma unroll
            for (int w = 0; w < 4; ++w) L += sm[w][j][hh] == -INFINITY ? 0.f : exp2f(sm[w][j][hh] - M) * sl[w][j][hh];
            rec[0] = M, rec[1] = L;
        }
    }
}

template <int NK, int NV>
static hipError_t step_go(const Gqa &g, const GqaStep &a, hipStream_t s) {
    const int splits = gqa_records(g), group = (int)(g.heads / g.kv_heads), nh = min(16, group);
    const size_t queries = g.maps * 16 * (NK * 32 + 4), outs = 4 * g.maps * nh * g.vdimp, lds = (queries > outs ? queries : outs) * sizeof(float);
    auto fn = g.maps == 2 ? k_gqa_step<NK, NV, 2> : k_gqa_step<NK, NV, 1>;
    if (lds > 65536) {
        const hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void *>(fn), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
        if (e != hipSuccess) return e;
    }
    hipLaunchKernelGGL(fn, dim3(splits, g.kv_heads * ((group + 15) / 16)), dim3(256), lds, s, g, a);
    return hipGetLastError();
}

hipError_t launch_gqa_step(const Gqa &g, const GqaStep &a, hipStream_t s) {
    if (!gqa_supported((int)g.dimp, (int)g.vdimp)) return hipErrorInvalidValue;
    if (g.dimp <= 64 && g.vdimp <= 64) return step_go<2, 4>(g, a, s);
    if (g.dimp <= 64 && g.vdimp <= 128) return step_go<2, 8>(g, a, s);
    if (g.dimp <= 128 && g.vdimp <= 128) return step_go<4, 8>(g, a, s);
    return step_go<8, 16>(g, a, s);
}

// ---- records -> output ------------------------------------------------------------------------------------------------
template <class TO>
__global__ __launch_bounds__(256) void k_gqa_merge(Gqa p, const int *pos_ptr, int q0, const float *scratch, TO *out, size_t ldo) {
    extern __shared__ __attribute__((aligned(16))) float part[];  // [maps][2][vdimp]
    static_assert(kGqaSplits == 128, "two records per lane of a wave");
    __shared__ float ws[2][kGqaSplits], sinv[2], slot[4];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, h = blockIdx.x, qi = blockIdx.z, maps = (int)p.maps, vdimp = (int)p.vdimp;
    const float z = p.gate ? gate_logit(p, qi, h, min(tid, vdimp - 1)) : 0.f, sink = p.sink ? p.sink[h] * kLog2e : -INFINITY;  // (ahead of the chain that starts with the position)
    const int used = gqa_range(p, *pos_ptr + q0 + qi).used;
    const size_t stride = kGqaRecHead + vdimp;
    const float *rec = scratch + ((size_t)qi * p.heads + h) * maps * kGqaSplits * stride;
    // 32 lanes of four columns; eight groups share maps and records.  Each group's first records are requested ahead of the weights.
    const int grp = tid >> 5, gm = maps == 2 ? grp & 1 : 0, gs = maps == 2 ? grp >> 1 : grp, gn = maps == 2 ? 4 : 8, i0 = (tid & 31) * 4;
    const float *vec = rec + (size_t)gm * kGqaSplits * stride + kGqaRecHead;
    constexpr int AHEAD = 4;
    f32x4 first[AHEAD];
#pragma unroll
    for (int e = 0; e < AHEAD; ++e) first[e] = *reinterpret_cast<const f32x4 *>(vec + min(gs + e * gn, used - 1) * stride + min(i0, vdimp - 4));
    if (wave < maps) {
        const float *r = rec + (size_t)wave * kGqaSplits * stride;
        float mv[2], lv[2];
#pragma unroll
        for (int e = 0; e < 2; ++e) {
            const int i = lane + 64 * e;
            mv[e] = i < used ? r[i * stride] : -INFINITY;
            lv[e] = i < used ? r[i * stride + 1] : 0.f;
        }
        const float M = fmaxf(sink, rows_max(row_max(fmaxf(mv[0], mv[1]))));
        float den = 0.f;
#pragma unroll
        for (int e = 0; e < 2; ++e) {
            const float w = lane + 64 * e < used ? exp2f(mv[e] - M) : 0.f;
            ws[wave][lane + 64 * e] = w;
            den += w * lv[e];
        }
        den = wave_sum(den) + (p.sink ? exp2f(sink - M) : 0.f);
        if (lane == 0) sinv[wave] = 1.0f / den;
    }
    __syncthreads();
    const float gate = p.gate ? activate(z, BITNET_HIP_ACT_SIGMOID) : 1.0f;
    for (int i = i0; i < vdimp; i += 128) {
        const float *r = vec + i;
        f32x4 acc = f32x4{0.f, 0.f, 0.f, 0.f};
        int k0 = gs;
        if (i == i0) {
#pragma unroll
            for (int e = 0; e < AHEAD; ++e) acc += ws[gm][gs + e * gn] * first[e];  // (weights past the last record are zero)
            k0 += AHEAD * gn;
        }
#pragma unroll 8
        for (int k = k0; k < used; k += gn) acc += ws[gm][k] * *reinterpret_cast<const f32x4 *>(r + k * stride);
        *reinterpret_cast<f32x4 *>(part + (size_t)grp * vdimp + i) = acc;
    }
    __syncthreads();
    float v = 0.f;
    const bool live = tid < vdimp;  // (vdimp <= 256; wider heads loop below)
    TO *dst = out + (size_t)qi * ldo + (size_t)h * vdimp;
    auto value = [&](int i) {
        if (maps == 1) {
            float t = 0.f;
#pragma unroll
            for (int k = 0; k < 8; ++k) t += part[k * vdimp + i];
            const float own = p.gate_columns && vdimp > 256 ? activate(gate_logit(p, qi, h, i), BITNET_HIP_ACT_SIGMOID) : gate;
            return t * (sinv[0] * own);
        }
        const float a = (part[i] + part[2 * vdimp + i]) + (part[4 * vdimp + i] + part[6 * vdimp + i]);
        const float b = (part[vdimp + i] + part[3 * vdimp + i]) + (part[5 * vdimp + i] + part[7 * vdimp + i]);
        return a * sinv[0] - p.lambda * (b * sinv[1]);
    };
    if (vdimp <= 256) {
        v = live ? value(tid) : 0.f;
        if (maps == 2) v *= gate * p.out_scale / sqrtf(group_sum<4>(v * v, slot) / (float)p.vdim + p.eps);
        if (live) st_act(dst, tid, v);
        return;
    }
    float ss = 0.f, f = 1.0f;
    for (int i = tid; i < vdimp; i += 256) v = value(i), ss += v * v;
    if (maps == 2) f = gate * p.out_scale / sqrtf(group_sum<4>(ss, slot) / (float)p.vdim + p.eps);
    for (int i = tid; i < vdimp; i += 256) st_act(dst, i, value(i) * f);
}

hipError_t launch_gqa_merge(const Gqa &g, const int *pos, int q0, int nq, const float *scratch, void *out, size_t ldo, int out_bf16, hipStream_t s) {
    const size_t lds = 8 * g.vdimp * sizeof(float);
    if (lds > 65536) return hipErrorInvalidValue;
    if (out_bf16)
        hipLaunchKernelGGL(k_gqa_merge<uint16_t>, dim3(g.heads, 1, nq), dim3(256), lds, s, g, pos, q0, scratch, (uint16_t *)out, ldo);
    else
        hipLaunchKernelGGL(k_gqa_merge<float>, dim3(g.heads, 1, nq), dim3(256), lds, s, g, pos, q0, scratch, (float *)out, ldo);
    return hipGetLastError();
}

// ---- prompt -----------------------------------------------------------------------------------------------------------
// One workgroup: one head, four waves; a wave holds two slots of 16 queries: both maps of one query tile, or two tiles of the only map.  Key tiles
// of 64 (every map's) and the values of the tile staged through registers into LDS one step ahead.
// FAR: with a distance penalty, gates per column, or both.
template <int NK, int NV, int MAPS, bool FAR>
__global__ __launch_bounds__(256, NV > 8 || NK > 4 ? 1 : 2) void k_gqa_prefill(Gqa p, const uint16_t *Q, size_t ldq, int n_ctx, int nq, uint16_t *out, size_t ldo, int n_qb) {
    extern __shared__ __attribute__((aligned(16))) uint8_t lds[];
    constexpr int SLOTS = 2, QW = 16 * SLOTS / MAPS, KS = NK * 64 + 16, VS = 64 * 2 + 16, NVL = NV / 2;
    uint8_t *lk = lds, *lv = lds + MAPS * 64 * KS;
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, r16 = lane & 15, g = lane >> 4;
    const int heads = (int)p.heads, dimp = (int)p.dimp, vdimp = (int)p.vdimp;
    // Consecutive workgroups go to the eight XCDs in turn.  Longest blocks first; an XCD keeps heads / 8 neighbouring heads of its own (their keys
    // and values stay in its L2), the heads left over move from XCD to XCD with the block so that all eight carry the same work.
    const int x = blockIdx.x & 7, rest = blockIdx.x >> 3, own = heads >> 3, left = heads & 7, per = own + (left ? 1 : 0);
    const int level = rest / per, slot = rest - level * per, r = (x + 8 * left - (level % 8) * left) & 7;
    if (slot == own && r >= left) return;
    const int h = slot < own ? x * own + slot : 8 * own + r, qb = n_qb - 1 - level;
    const int kv = h / (int)(p.heads / p.kv_heads), q0 = qb * 4 * QW, pos0 = n_ctx - nq, qw = q0 + wave * QW;
    bf16x8 qf[SLOTS][NK];
    int qpos[SLOTS], qfirst[SLOTS];
#pragma unroll
    for (int t = 0; t < SLOTS; ++t) {
        const int tile = t / MAPS, map = t % MAPS, qi = min(qw + tile * 16 + r16, nq - 1);
        qpos[t] = pos0 + qw + tile * 16 + r16;
        qfirst[t] = gqa_first(p, qpos[t]);
        const uint16_t *q = Q + (size_t)qi * ldq + (size_t)(h * MAPS + map) * dimp;
#pragma unroll
        for (int kk = 0; kk < NK; ++kk) {
            u32x4 v = *reinterpret_cast<const u32x4 *>(q + min(kk * 32, dimp - 32) + g * 8);
            const uint32_t keep = kk * 32 < dimp ? 0xffffffffu : 0u;
            qf[t][kk] = __builtin_bit_cast(bf16x8, u32x4{v.x & keep, v.y & keep, v.z & keep, v.w & keep});
        }
    }
    f32x4 o[NV][SLOTS];
    float m[SLOTS], l[SLOTS];
#pragma unroll
    for (int t = 0; t < SLOTS; ++t) {
        // (finite: with chunks a tile may hold no key that a query sees; the sink counts once per query, four lanes share one)
        m[t] = MAPS == 1 && p.sink ? p.sink[h] * kLog2e : -1e30f, l[t] = MAPS == 1 && p.sink && g == 0 ? 1.0f : 0.f;
#pragma unroll
        for (int v = 0; v < NV; ++v) o[v][t] = f32x4{0.f, 0.f, 0.f, 0.f};
    }
    const uint16_t *K = (const uint16_t *)p.kcache + (size_t)kv * MAPS * p.capacity * dimp, *V = (const uint16_t *)p.vcache + (size_t)kv * vdimp * p.capacity;
    u32x4 kreg[MAPS][NK], vreg[NVL];
    const unsigned koff = (unsigned)((tid >> 2) * dimp * 2 + (tid & 3) * 16);
    const size_t voff = (size_t)(tid >> 3) * p.capacity * 2 + (tid & 7) * 16;
#pragma unroll
    for (int j = 0; j < NVL; ++j) vreg[j] = u32x4{0u, 0u, 0u, 0u};
    auto fetch = [&](int key0) {  // (whole tiles: the capacity is a multiple of 64)
#pragma unroll
        for (int mp = 0; mp < MAPS; ++mp) {
            const char *kb = (const char *)(K + ((size_t)mp * p.capacity + key0) * dimp);
#pragma unroll
            for (int j = 0; j < NK; ++j) kreg[mp][j] = *reinterpret_cast<const u32x4 *>(kb + min(j * 64, dimp * 2 - 64) + koff);
        }
        const char *vb = (const char *)(V + key0);
#pragma unroll
        for (int j = 0; j < NVL; ++j)
            if (j * 32 < vdimp) vreg[j] = *reinterpret_cast<const u32x4 *>(vb + (size_t)j * 64 * p.capacity + voff);
    };
    const int n_tiles = (min(n_ctx, pos0 + q0 + 4 * QW) + 63) / 64;
    const FarPenalty far = far_penalty(p, h);
    // tiles from the first key of the workgroup's first query on; a wave leaves out what lies ahead of its own first key
    const int t_first = gqa_first(p, pos0 + q0) >> 6, w_first = gqa_first(p, pos0 + qw), w_last = gqa_first(p, pos0 + qw + QW - 1);
    fetch(t_first * 64);
    for (int kt0 = t_first; kt0 < n_tiles; ++kt0) {
        const int key0 = kt0 * 64;
        __syncthreads();
#pragma unroll
        for (int mp = 0; mp < MAPS; ++mp)
#pragma unroll
            for (int j = 0; j < NK; ++j) *reinterpret_cast<u32x4 *>(lk + (mp * 64 + (tid >> 2)) * KS + j * 64 + (tid & 3) * 16) = kreg[mp][j];
#pragma unroll
        for (int j = 0; j < NVL; ++j) *reinterpret_cast<u32x4 *>(lv + ((tid >> 3) + 32 * j) * VS + (tid & 7) * 16) = vreg[j];
        __syncthreads();
        if (kt0 + 1 < n_tiles) fetch(key0 + 64);
        if (key0 > pos0 + qw + QW - 1 || key0 + 63 < w_first) continue;  // no key of the tile is seen by this wave's queries
        f32x4 s[4][SLOTS];
#pragma unroll
        for (int kt = 0; kt < 4; ++kt) {
#pragma unroll
            for (int t = 0; t < SLOTS; ++t) s[kt][t] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int kk = 0; kk < NK; ++kk)
#pragma unroll
                for (int t = 0; t < SLOTS; ++t) {
                    const bf16x8 a = *reinterpret_cast<const bf16x8 *>(lk + ((t % MAPS) * 64 + kt * 16 + r16) * KS + kk * 64 + g * 16);
                    s[kt][t] = mfma_bf16(a, qf[t][kk], s[kt][t]);
                }
        }
        if (FAR && p.far_weight)
#pragma unroll
            for (int t = 0; t < SLOTS; ++t)
#pragma unroll
                for (int kt = 0; kt < 4; ++kt)
#pragma unroll
                    for (int i = 0; i < 4; ++i) s[kt][t][i] = nearer(s[kt][t][i], far, qpos[t] - (key0 + kt * 16 + g * 4 + i));
        if (key0 + 63 > pos0 + qw)  // the diagonal
#pragma unroll
            for (int t = 0; t < SLOTS; ++t)
#pragma unroll
                for (int kt = 0; kt < 4; ++kt)
#pragma unroll
                    for (int i = 0; i < 4; ++i) s[kt][t][i] = key0 + kt * 16 + g * 4 + i > qpos[t] ? -INFINITY : s[kt][t][i];
        if (key0 < w_last)  // an earlier chunk of some of the queries
#pragma unroll
            for (int t = 0; t < SLOTS; ++t)
#pragma unroll
                for (int kt = 0; kt < 4; ++kt)
#pragma unroll
                    for (int i = 0; i < 4; ++i) s[kt][t][i] = key0 + kt * 16 + g * 4 + i < qfirst[t] ? -INFINITY : s[kt][t][i];
        float mn[SLOTS];
        bool grows = false;
#pragma unroll
        for (int t = 0; t < SLOTS; ++t) {
            float mx = fmaxf(fmaxf(s[0][t][0], s[0][t][1]), fmaxf(s[0][t][2], s[0][t][3]));
#pragma unroll
            for (int kt = 1; kt < 4; ++kt) mx = fmaxf(mx, fmaxf(fmaxf(s[kt][t][0], s[kt][t][1]), fmaxf(s[kt][t][2], s[kt][t][3])));
            mn[t] = fmaxf(m[t], rows_max(mx) * kLog2e);
            grows = grows || mn[t] > m[t];
        }
        if (__any(grows)) {
#pragma unroll
            for (int t = 0; t < SLOTS; ++t) {
                const float al = __builtin_amdgcn_exp2f(m[t] - mn[t]);
                m[t] = mn[t];
                l[t] *= al;
#pragma unroll
                for (int v = 0; v < NV; ++v) o[v][t] *= al;
            }
        }
        SplitFrag pf[2][SLOTS];
#pragma unroll
        for (int ks = 0; ks < 2; ++ks)
#pragma unroll
            for (int t = 0; t < SLOTS; ++t) {
                f32x4 w[2];
#pragma unroll
                for (int j = 0; j < 2; ++j) {
#pragma unroll
                    for (int i = 0; i < 4; ++i) w[j][i] = __builtin_amdgcn_exp2f(fmaf(s[2 * ks + j][t][i], kLog2e, -m[t]));
                    l[t] += (w[j][0] + w[j][1]) + (w[j][2] + w[j][3]);
                }
                pf[ks][t] = split8(w[0], w[1]);
            }
#pragma unroll
        for (int v = 0; v < NV; ++v)
#pragma unroll
            for (int ks = 0; ks < 2; ++ks) {
                const uint8_t *row = lv + (v * 16 + r16) * VS + ks * 64 + g * 8;
                const u32x2 a0 = *reinterpret_cast<const u32x2 *>(row), a1 = *reinterpret_cast<const u32x2 *>(row + 32);
                const bf16x8 a = __builtin_bit_cast(bf16x8, u32x4{a0.x, a0.y, a1.x, a1.y});
#pragma unroll
                for (int t = 0; t < SLOTS; ++t) {
                    o[v][t] = mfma_bf16(a, pf[ks][t].hi, o[v][t]);
                    o[v][t] = mfma_bf16(a, pf[ks][t].lo, o[v][t]);
                }
            }
    }
    float inv[SLOTS], gate[SLOTS / MAPS];
#pragma unroll
    for (int t = 0; t < SLOTS / MAPS; ++t) gate[t] = 1.0f;
#pragma unroll
    for (int t = 0; t < SLOTS; ++t) inv[t] = 1.0f / rows_sum(l[t]);
    if (p.gate && !(FAR && p.gate_columns))
#pragma unroll
        for (int t = 0; t < SLOTS / MAPS; ++t) gate[t] = activate(gate_logit(p, min(qw + t * 16 + r16, nq - 1), h, 0), BITNET_HIP_ACT_SIGMOID);
    if (MAPS == 2) {
        float ss = 0.f;
#pragma unroll
        for (int v = 0; v < NV; ++v) {
            o[v][0] = o[v][0] * inv[0] - (p.lambda * inv[1]) * o[v][1];
            ss += (o[v][0].x * o[v][0].x + o[v][0].y * o[v][0].y) + (o[v][0].z * o[v][0].z + o[v][0].w * o[v][0].w);
        }
        inv[0] = p.out_scale / sqrtf(rows_sum(ss) / (float)p.vdim + p.eps);
    }
#pragma unroll
    for (int t = 0; t < SLOTS / MAPS; ++t) {
        const int qi = qw + t * 16 + r16;
        if (qi >= nq) continue;
        uint16_t *dst = out + (size_t)qi * ldo + (size_t)h * vdimp + g * 4;
#pragma unroll
        for (int v = 0; v < NV; ++v)
            if (v * 16 < vdimp) {
                f32x4 q = o[v][t] * (inv[t] * gate[t]);
                if (FAR && p.gate_columns) {
                    float z[4];
#pragma unroll
                    for (int i = 0; i < 4; ++i) z[i] = gate_logit(p, qi, h, v * 16 + g * 4 + i);
#pragma unroll
                    for (int i = 0; i < 4; ++i) q[i] *= __builtin_amdgcn_rcpf(1.0f + __expf(-z[i]));
                }
                *reinterpret_cast<bf16x4 *>(dst + v * 16) = bf16x4{(__bf16)q.x, (__bf16)q.y, (__bf16)q.z, (__bf16)q.w};
            }
    }
}

template <int NK, int NV>
static hipError_t gqa_prefill_go(const Gqa &g, const uint16_t *q, size_t ldq, int n_ctx, int nq, uint16_t *out, size_t ldo, hipStream_t s) {
    const int rows = g.maps == 2 ? 64 : 128, n_qb = (nq + rows - 1) / rows;
    const size_t lds = (size_t)g.maps * 64 * (NK * 64 + 16) + (size_t)NV * 16 * (64 * 2 + 16);
    auto fn = g.maps == 2 ? k_gqa_prefill<NK, NV, 2, false> : g.far_weight || g.gate_columns ? k_gqa_prefill<NK, NV, 1, true> : k_gqa_prefill<NK, NV, 1, false>;
    if (lds > 65536) {
        const hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void *>(fn), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
        if (e != hipSuccess) return e;
    }
    hipLaunchKernelGGL(fn, dim3(8 * ((g.heads + 7) / 8) * n_qb), dim3(256), lds, s, g, q, ldq, n_ctx, nq, out, ldo, n_qb);
    return hipGetLastError();
}

hipError_t launch_gqa_prefill(const Gqa &g, const uint16_t *q, size_t ldq, int n_ctx, int nq, uint16_t *out, size_t ldo, hipStream_t s) {
    if (!gqa_supported((int)g.dimp, (int)g.vdimp)) return hipErrorInvalidValue;
    if (g.dimp <= 64 && g.vdimp <= 64) return gqa_prefill_go<2, 4>(g, q, ldq, n_ctx, nq, out, ldo, s);
    if (g.dimp <= 64 && g.vdimp <= 128) return gqa_prefill_go<2, 8>(g, q, ldq, n_ctx, nq, out, ldo, s);
    if (g.dimp <= 128 && g.vdimp <= 128) return gqa_prefill_go<4, 8>(g, q, ldq, n_ctx, nq, out, ldo, s);
    return gqa_prefill_go<8, 16>(g, q, ldq, n_ctx, nq, out, ldo, s);
}

}  // namespace bitnet_hip
