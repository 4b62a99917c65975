// kernels_experts.hip -- mixture of experts (gfx950): the choice of a token's experts, the row lists of the grouped products
// (kernels_dense.hip) and the matrix-vector products of the decode step.
//
// The router's logits, scores and weights are f32.  A prompt's choices become slots: an expert's slots lie side by side, cut into tiles of rows
// (expert, first slot, slots); a slot's token is its activation row on the way up, the slot itself is the row on the way down.
#include "dense.hpp"

namespace bitnet_hip {

// LT lanes choose one token's experts: lane k < top of them receives the k-th one and its weight.  A lane holds PL neighbouring experts, so that
// among equal scores the lowest lane has the lowest index.
template <int LT>
__device__ __forceinline__ float token_max(float v) {
    v = row_max(v);
    return LT == 64 ? rows_max(v) : v;
}
template <int LT>
__device__ __forceinline__ float token_sum(float v) {
    v = row_sum(v);
    return LT == 64 ? rows_sum(v) : v;
}

template <int LT, int PL>
__device__ __forceinline__ void choose_load(const float *z, int experts, float (&s)[PL]) {
    const int l = threadIdx.x & (LT - 1);
#pragma unroll
    for (int j = 0; j < PL; ++j) s[j] = l * PL + j < experts ? z[l * PL + j] : -INFINITY;
}

// the two largest of the pairs (a1 >= a2) and (b1 >= b2)
__device__ __forceinline__ void two_largest(float &a1, float &a2, float b1, float b2) {
    const float low = fmaxf(fminf(a1, b1), fmaxf(a2, b2));
    a1 = fmaxf(a1, b1), a2 = low;
}

// Choice scores s of a token: those of the groups that are not among the best become minus infinity.
template <int LT, int PL>
__device__ __forceinline__ void keep_groups(float (&s)[PL], const Router &r) {
    const int groups = (int)r.groups, keep = (int)r.keep, size = (int)r.experts / groups;
    const int lane = threadIdx.x & 63, l = lane & (LT - 1), base = lane & ~(LT - 1);
    auto worth = [&](float a1, float a2) { return size > 1 ? a1 + a2 : a1; };
    const int span = size / PL;  // lanes of a group, where it fills them and they are a power of two
    if (span * PL == size && (span & (span - 1)) == 0) {
        float a1 = -INFINITY, a2 = -INFINITY;
#pragma unroll
        for (int j = 0; j < PL; ++j) two_largest(a1, a2, s[j], -INFINITY);
        for (int off = 1; off < span; off <<= 1) {
            const float b1 = __shfl_xor(a1, off, 64), b2 = __shfl_xor(a2, off, 64);
            two_largest(a1, a2, b1, b2);
        }
        const float w = worth(a1, a2);
        const int mine = l / span;
        int ahead = 0;
        for (int g = 0; g < groups; ++g) {
            const float o = __shfl(w, base + g * span, 64);
            ahead += o > w || (o == w && g < mine);
        }
#pragma unroll
        for (int j = 0; j < PL; ++j) s[j] = ahead < keep ? s[j] : -INFINITY;
        return;
    }
    // groups that do not: each one's worth by itself; a lane keeps the worth of every expert's group
    float w[PL];
    int ahead[PL];
#pragma unroll
    for (int j = 0; j < PL; ++j) w[j] = -INFINITY, ahead[j] = 0;
    auto of_group = [&](int g) {
        float a1 = -INFINITY, a2 = -INFINITY;
#pragma unroll
        for (int j = 0; j < PL; ++j) {
            const int e = l * PL + j;
            two_largest(a1, a2, e >= g * size && e < (g + 1) * size ? s[j] : -INFINITY, -INFINITY);
        }
        for (int off = 1; off < LT; off <<= 1) {
            const float b1 = __shfl_xor(a1, off, 64), b2 = __shfl_xor(a2, off, 64);
            two_largest(a1, a2, b1, b2);
        }
        return worth(a1, a2);
    };
    for (int g = 0; g < groups; ++g) {
        const float o = of_group(g);
#pragma unroll
        for (int j = 0; j < PL; ++j) w[j] = (l * PL + j) / size == g ? o : w[j];
    }
    for (int g = 0; g < groups; ++g) {
        const float o = of_group(g);
#pragma unroll
        for (int j = 0; j < PL; ++j) ahead[j] += o > w[j] || (o == w[j] && g < (l * PL + j) / size);
    }
#pragma unroll
    for (int j = 0; j < PL; ++j) s[j] = ahead[j] < keep ? s[j] : -INFINITY;
}

template <int LT, int PL, bool GROUPED>
__device__ __forceinline__ void choose(float (&s)[PL], const Router &r, int &id, float &weight) {
    const int experts = (int)(r.experts + r.identity), top = (int)r.top;
    const int lane = threadIdx.x & 63, l = lane & (LT - 1), base = lane & ~(LT - 1);
    if (r.sigmoid) {
#pragma unroll
        for (int j = 0; j < PL; ++j) s[j] = l * PL + j < experts ? 1.0f / (1.0f + expf(-s[j])) : -INFINITY;
    } else {
        float m = -INFINITY, sum = 0.f;
#pragma unroll
        for (int j = 0; j < PL; ++j) m = fmaxf(m, s[j]);
        m = token_max<LT>(m);
#pragma unroll
        for (int j = 0; j < PL; ++j) {
            s[j] = s[j] == -INFINITY ? 0.f : expf(s[j] - m);
            sum += s[j];
        }
        sum = token_sum<LT>(sum);
#pragma unroll
        for (int j = 0; j < PL; ++j) s[j] = l * PL + j < experts ? s[j] / sum : -INFINITY;  // (-infinity: not there, or taken)
    }
    float score[PL];  // without the correction
#pragma unroll
    for (int j = 0; j < PL; ++j) {
        score[j] = s[j];
        if (r.correction) s[j] += r.correction[min(l * PL + j, experts - 1)];
    }
    if (GROUPED) keep_groups<LT, PL>(s, r);
    id = 0, weight = 0.f;
    float chosen = 0.f;
    for (int k = 0; k < top; ++k) {
        float best = -INFINITY;
        int at = 0;
#pragma unroll
        for (int j = 0; j < PL; ++j)
            if (s[j] > best) best = s[j], at = j;
        const float w = token_max<LT>(best);
        unsigned long long who = __ballot(best == w) >> base;
        if (LT < 64) who &= (1ull << LT) - 1;
        const int winner = who ? __builtin_ctzll(who) : 0;  // (no score compares equal to itself if a logit is not a number)
        const int mine = l * PL + at;
        const int e = min(LT == 64 ? __builtin_amdgcn_readlane(mine, winner) : __shfl(mine, base + winner, 64), experts - 1);
        if (l == k) id = e, weight = w;
        chosen += w;
        if (l == winner)
#pragma unroll
            for (int j = 0; j < PL; ++j)
                if (j == at) s[j] = -INFINITY;
    }
    if (r.correction) {  // the scores of what was chosen
        float w = 0.f;
#pragma unroll
        for (int j = 0; j < PL; ++j) {
            const float t = __shfl(score[j], base + id / PL, 64);
            w = id % PL == j ? t : w;
        }
        weight = l < top ? w : 0.f;
        chosen = token_sum<LT>(weight);
    }
    weight = (r.raw ? weight : weight / (chosen + 1e-20f)) * r.scale;
}

// ---- a prompt's choices -----------------------------------------------------------------------------------------------
constexpr int kRouteTokens = 32;  // per workgroup; its choices are counted in LDS first

template <int LT, int PL, bool GROUPED>
__global__ __launch_bounds__(256) void k_route(const float *__restrict__ z, size_t ldz, Router r, ExpertsPlan p) {
    __shared__ int hist[kMaxExperts];
    const int tid = threadIdx.x, grp = tid / LT, l = tid & (LT - 1), experts = (int)p.experts, outputs = (int)(r.experts + r.identity), top = (int)p.top, m = (int)p.m;
    constexpr int PER = kRouteTokens * LT / 256;  // (top <= LT)
    const int t0 = blockIdx.x * kRouteTokens + grp * PER;
    float s[PER][PL];
#pragma unroll
    for (int i = 0; i < PER; ++i) choose_load<LT, PL>(z + (size_t)min(t0 + i, m - 1) * ldz, outputs, s[i]);
    for (int e = tid; e < experts; e += 256) hist[e] = 0;
    __syncthreads();
    int id[PER], rank[PER];
#pragma unroll
    for (int i = 0; i < PER; ++i) {
        float w;
        choose<LT, PL, GROUPED>(s[i], r, id[i], w);
        rank[i] = 0;
        if (t0 + i < m && l < top) {
            if (id[i] < experts) rank[i] = atomicAdd(&hist[id[i]], 1);
            p.ids[(size_t)(t0 + i) * top + l] = id[i];
            p.weights[(size_t)(t0 + i) * top + l] = w;
        }
    }
    __syncthreads();
    for (int e = tid; e < experts; e += 256) {
        const int c = hist[e];
        hist[e] = c ? atomicAdd(&p.counts[e], c) : 0;
    }
    __syncthreads();
#pragma unroll
    for (int i = 0; i < PER; ++i)
        if (t0 + i < m && l < top) p.slots[(size_t)(t0 + i) * top + l] = id[i] < experts ? rank[i] + hist[id[i]] : -1;  // within its expert so far
}

// first slot and tiles of every expert; the counts are left at zero for the next portion
__global__ __launch_bounds__(1024) void k_route_tiles(ExpertsPlan p) {
    __shared__ int2 sums[kMaxExperts];
    const int e = threadIdx.x, experts = (int)p.experts, tile = (int)p.tile;
    const int count = e < experts ? p.counts[e] : 0, tiles = (count + tile - 1) / tile;
    sums[e] = make_int2(count, tiles);
    __syncthreads();
    for (int off = 1; off < kMaxExperts; off <<= 1) {
        const int2 mine = sums[e], other = e >= off ? sums[e - off] : make_int2(0, 0);
        __syncthreads();
        sums[e] = make_int2(mine.x + other.x, mine.y + other.y);
        __syncthreads();
    }
    if (e < experts) {
        const int first = sums[e].x - count, t0 = sums[e].y - tiles;
        p.offsets[e] = first;
        p.counts[e] = 0;
        for (int i = 0; i < tiles; ++i)
            if (t0 + i < (int)p.max_tiles) reinterpret_cast<int4 *>(p.tiles)[t0 + i] = make_int4(e, first + i * tile, min(tile, count - i * tile), 0);
    }
    if (e == 0) *p.n_tiles = min(sums[kMaxExperts - 1].y, (int)p.max_tiles);
}

__global__ __launch_bounds__(256) void k_route_slots(ExpertsPlan p) {
    const int i = blockIdx.x * 256 + threadIdx.x;
    if (i >= (int)(p.m * p.top)) return;
    if (p.ids[i] >= (int)p.experts) return;  // (an identity expert)
    const int s = p.offsets[p.ids[i]] + p.slots[i];
    p.slots[i] = s;
    p.tokens[s] = i / (int)p.top;
}

hipError_t launch_experts_route(const float *logits, size_t ldz, const Router &r, const ExpertsPlan &p, hipStream_t s) {
    const bool row = p.top <= 16;  // sixteen lanes per token
    const int e = (int)(r.experts + r.identity);
    auto pick = [&](auto any, auto grouped) { return r.groups ? grouped : any; };
    auto fn = row && e <= 16    ? pick(k_route<16, 1, false>, k_route<16, 1, true>)
              : row && e <= 64  ? pick(k_route<16, 4, false>, k_route<16, 4, true>)
              : row && e <= 128 ? pick(k_route<16, 8, false>, k_route<16, 8, true>)
              : e <= 256        ? pick(k_route<64, 4, false>, k_route<64, 4, true>)
                                : pick(k_route<64, 16, false>, k_route<64, 16, true>);
    hipLaunchKernelGGL(fn, dim3((p.m + kRouteTokens - 1) / kRouteTokens), dim3(256), 0, s, logits, ldz, r, p);
    hipLaunchKernelGGL(k_route_tiles, dim3(1), dim3(1024), 0, s, p);
    hipLaunchKernelGGL(k_route_slots, dim3((p.m * p.top + 255) / 256), dim3(256), 0, s, p);
    return hipGetLastError();
}

// ---- one token --------------------------------------------------------------------------------------------------------
// Both products in the manner of k_dense_gemv: LPR lanes per row, 16 bytes of weights per lane and chunk of LPR * 8 columns, R rows x U chunks in
// flight, the input vector in LDS with every segment padded to whole chunks.
constexpr int kStage = 4;  // sixteen-byte loads in flight per thread while the vector is staged (rows and segments start on 16 bytes)

template <int R>
__device__ __forceinline__ void multiply8(const u32x4 (&w)[R], const float *x, float (&acc)[R]) {
    const f32x4 x0 = *reinterpret_cast<const f32x4 *>(x), x1 = *reinterpret_cast<const f32x4 *>(x + 4);
#pragma unroll
    for (int r = 0; r < R; ++r) {
        acc[r] = fmaf(x0.x, __builtin_bit_cast(float, w[r].x << 16), acc[r]);
        acc[r] = fmaf(x0.y, __builtin_bit_cast(float, w[r].x & 0xffff0000u), acc[r]);
        acc[r] = fmaf(x0.z, __builtin_bit_cast(float, w[r].y << 16), acc[r]);
        acc[r] = fmaf(x0.w, __builtin_bit_cast(float, w[r].y & 0xffff0000u), acc[r]);
        acc[r] = fmaf(x1.x, __builtin_bit_cast(float, w[r].z << 16), acc[r]);
        acc[r] = fmaf(x1.y, __builtin_bit_cast(float, w[r].z & 0xffff0000u), acc[r]);
        acc[r] = fmaf(x1.z, __builtin_bit_cast(float, w[r].w << 16), acc[r]);
        acc[r] = fmaf(x1.w, __builtin_bit_cast(float, w[r].w & 0xffff0000u), acc[r]);
    }
}
template <int LPR>
__device__ __forceinline__ float lanes_sum(float v) {
    v = row_sum(v);
    if (LPR == 64) return rows_sum(v);
    if (LPR == 32) {
        float w = v;
        swap_rows16(v, w);
        v += w;
    }
    return v;
}

struct UpK {
    ExpertsUp a;
    int kp, groups;
};

template <int LPR, int R, int U, int PL, bool GROUPED>
__global__ __launch_bounds__(256) void k_experts_up(UpK p) {
    extern __shared__ __attribute__((aligned(16))) float xs[];
    const ExpertsUp &a = p.a;
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, b = blockIdx.y, sub = lane / LPR, l = lane % LPR;
    constexpr int G = 64 / LPR, CH = LPR * 8;
    float z[PL];
    choose_load<64, PL>(a.logits, (int)(a.r.experts + a.r.identity), z);
    f32x4 xv[kStage];
    auto load = [&](int i0) {
#pragma unroll
        for (int j = 0; j < kStage; ++j) xv[j] = reinterpret_cast<const f32x4 *>(a.x)[min(i0 + 256 * j, a.cols / 4 - 1)];
    };
    auto store = [&](int i0) {
#pragma unroll
        for (int j = 0; j < kStage; ++j) {
            const int i = i0 + 256 * j;
            if (i < p.kp / 4) reinterpret_cast<f32x4 *>(xs)[i] = i < a.cols / 4 ? xv[j] : f32x4{0.f, 0.f, 0.f, 0.f};
        }
    };
    load(tid);
    int mine;
    float weight;
    choose<64, PL, GROUPED>(z, a.r, mine, weight);
    // member b of the launch takes the b-th chosen expert that is no identity
    const unsigned long long real = __ballot(lane < (int)a.r.top && mine < (int)a.r.experts);
    const int n_real = __popcll(real);
    if (blockIdx.x == 0 && b == 0 && wave == 0) {
        const int rank = __popcll(real & ((1ull << lane) - 1));
        if (real >> lane & 1) a.ids[rank] = mine;
        if (lane >= n_real && lane < (int)a.r.top) a.ids[lane] = -1;
        if (a.identity) {
            const float sum = wave_sum(lane < (int)a.r.top && mine >= (int)a.r.experts ? weight : 0.f);
            if (lane == 0) *a.identity = sum;
        }
    }
    if (b >= n_real) return;
    int from = b;  // the b-th lane of those
    if (n_real < (int)a.r.top) {
        unsigned long long left = real;
        for (int i = 0; i < b; ++i) left &= left - 1;
        from = __builtin_ctzll(left);
    }
    const int e = __builtin_amdgcn_readlane(mine, from);
    const float scale = __builtin_bit_cast(float, __builtin_amdgcn_readlane(__builtin_bit_cast(int, weight), from));
    const uint16_t *wb = a.w + (size_t)e * a.rows * a.ld;
    const int last = a.cols - 8;
    u32x4 w[U][R];
    auto fetch = [&](int grp, int k0) {
#pragma unroll
        for (int r = 0; r < R; ++r) {
            const uint16_t *wr = wb + (size_t)min((grp * G + sub) * R + r, a.rows - 1) * a.ld;
#pragma unroll
            for (int u = 0; u < U; ++u) w[u][r] = __builtin_nontemporal_load(reinterpret_cast<const u32x4 *>(wr + min(k0 + (u * LPR + l) * 8, last)));
        }
    };
    int g = blockIdx.x * 4 + wave;
    if (g < p.groups) fetch(g, 0);
    store(tid);
    for (int i0 = tid + 256 * kStage; i0 < p.kp / 4; i0 += 256 * kStage) {
        load(i0);
        store(i0);
    }
    __syncthreads();
    const int n_wg = gridDim.x;
    for (; g < p.groups; g += n_wg * 4) {
        float acc[R];
#pragma unroll
        for (int r = 0; r < R; ++r) acc[r] = 0.f;
        for (int k0 = 0; k0 < p.kp; k0 += CH * U) {
            u32x4 c[U][R];
#pragma unroll
            for (int u = 0; u < U; ++u)
#pragma unroll
                for (int r = 0; r < R; ++r) c[u][r] = w[u][r];
            if (k0 + CH * U < p.kp)
                fetch(g, k0 + CH * U);
            else if (g + n_wg * 4 < p.groups)
                fetch(g + n_wg * 4, 0);
#pragma unroll
            for (int u = 0; u < U; ++u) multiply8<R>(c[u], xs + k0 + (u * LPR + l) * 8, acc);
        }
        if (R > 1 && a.gated) {
#pragma unroll
            for (int r = 0; r + 1 < R; r += 2) {
                const float v = lanes_sum<LPR>(acc[r]), u = lanes_sum<LPR>(acc[r + 1]);
                const int row = (g * G + sub) * R + r;
                if (l == 0 && row < a.rows) a.y[(size_t)b * a.ldy + (row >> 1)] = scale * (activate(v, a.act) * u);
            }
        } else {
#pragma unroll
            for (int r = 0; r < R; ++r) {
                const float v = lanes_sum<LPR>(acc[r]);
                const int row = (g * G + sub) * R + r;
                if (l == 0 && row < a.rows) a.y[(size_t)b * a.ldy + row] = scale * activate(v, a.act);
            }
        }
    }
}

struct OutK {
    ExpertsOut a;
    int c0, ce, chunks;  // chunks of the first segment, of an expert's, of all (rounded up to whole steps)
    unsigned magic;      // ceil(2^20 / ce)
    int groups;
};

template <int LPR, int R, int U>
__global__ __launch_bounds__(256) void k_experts_out(OutK p) {
    extern __shared__ __attribute__((aligned(16))) float xs[];
    const ExpertsOut &a = p.a;
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, sub = lane / LPR, l = lane % LPR;
    constexpr int G = 64 / LPR, CH = LPR * 8;
    const int ids = lane < a.top ? a.ids[lane] : -1, n_real = __popcll(__ballot(ids >= 0)), end = p.c0 + n_real * p.ce;
    u32x4 w[U][R];
    auto fetch = [&](int grp, int chunk0) {
#pragma unroll
        for (int u = 0; u < U; ++u) {
            const int c = chunk0 + u, x = max(c - p.c0, 0);
            const int q = min((int)((unsigned)x * p.magic >> 20), max(n_real - 1, 0)), e = max(__builtin_amdgcn_readlane(ids, q), 0);
            const bool first = c < p.c0;
            const uint16_t *base = first ? a.w0 : a.w1 + (size_t)e * a.rows * a.ld1;
            const int ld = first ? a.ld0 : a.ld1, col = min((first ? c : x - q * p.ce) * CH + l * 8, (first ? a.cols0 : a.cols1) - 8);
#pragma unroll
            for (int r = 0; r < R; ++r)
                w[u][r] = __builtin_nontemporal_load(reinterpret_cast<const u32x4 *>(base + (size_t)min((grp * G + sub) * R + r, a.rows - 1) * ld + col));
        }
    };
    int g = blockIdx.x * 4 + wave;
    if (g < p.groups) fetch(g, 0);
    const int steps = (end + U - 1) / U * U, total = steps * CH / 4;  // (identity experts have no columns)
    const float through = a.identity ? *a.identity : 0.f, scale0 = a.x0_scale ? *a.x0_scale : 1.0f;
    constexpr int AH = 12;
    for (int i0 = tid; i0 < total; i0 += 256 * AH) {
        f32x4 v[AH];
        float in[AH];  // zero: past a segment's columns
#pragma unroll
        for (int j = 0; j < AH; ++j) {
            const int i = i0 + 256 * j, c = i / (CH / 4), x = max(c - p.c0, 0), q = min((int)((unsigned)x * p.magic >> 20), max(n_real - 1, 0));
            const bool first = c < p.c0;
            const int col = (first ? i : i - (p.c0 + q * p.ce) * (CH / 4)) * 4, cols = first ? a.cols0 : a.cols1;
            in[j] = col < cols && c < end ? (first ? scale0 : 1.0f) : 0.f;
            v[j] = *reinterpret_cast<const f32x4 *>((first ? a.x0 : a.x1 + (size_t)q * a.ldx1) + min(col, cols - 4));
        }
#pragma unroll
        for (int j = 0; j < AH; ++j)
            if (i0 + 256 * j < total) reinterpret_cast<f32x4 *>(xs)[i0 + 256 * j] = in[j] != 0.f ? in[j] * v[j] : f32x4{0.f, 0.f, 0.f, 0.f};
    }
    __syncthreads();
    const int n_wg = gridDim.x;
    for (; g < p.groups; g += n_wg * 4) {
        float acc[R], more[R];
#pragma unroll
        for (int r = 0; r < R; ++r) {
            const int row = min((g * G + sub) * R + r, a.rows - 1);
            acc[r] = 0.f;
            more[r] = (a.bias ? a.bias[row] : 0.f) + (a.identity ? through * a.input[row] : 0.f);
        }
        for (int c0 = 0; c0 < steps; c0 += U) {
            u32x4 c[U][R];
#pragma unroll
            for (int u = 0; u < U; ++u)
#pragma unroll
                for (int r = 0; r < R; ++r) c[u][r] = w[u][r];
            if (c0 + U < steps)
                fetch(g, c0 + U);
            else if (g + n_wg * 4 < p.groups)
                fetch(g + n_wg * 4, 0);
#pragma unroll
            for (int u = 0; u < U; ++u) multiply8<R>(c[u], xs + (c0 + u) * CH + l * 8, acc);
        }
#pragma unroll
        for (int r = 0; r < R; ++r) {
            const float v = lanes_sum<LPR>(acc[r]);
            const int row = (g * G + sub) * R + r;
            if (l == 0 && row < a.rows) a.y[row] = v + more[r];
        }
    }
}

// workgroups of a product: all of them at once up to three per CU, whole rounds of row groups beyond
static int gemv_grid(int groups, int share) {
    int n = (groups + 3) / 4;
    const int cap = share > 1 ? (768 + share - 1) / share : 768;
    if (n > cap) {
        const int rounds = (n + cap - 1) / cap;
        n = (n + rounds - 1) / rounds;
    }
    return n;
}

template <int LPR, int R, bool GROUPED>
static hipError_t up_go(const ExpertsUp &a, int chunks, hipStream_t s) {
    UpK k;
    k.a = a;
    const int u = chunks % 5 == 0 ? 5 : chunks >= 3 ? 3 : chunks;
    k.kp = (chunks + u - 1) / u * u * LPR * 8;
    k.groups = (a.rows + 64 / LPR * R - 1) / (64 / LPR * R);
    if ((size_t)k.kp * 4 > 150 * 1024) return hipErrorInvalidValue;
    const int outputs = (int)(a.r.experts + a.r.identity), top = (int)a.r.top;
    auto pick = [&](auto f64, auto f256, auto f1024) { return outputs <= 64 ? f64 : outputs <= 256 ? f256 : f1024; };
    auto fn = u == 1   ? pick(k_experts_up<LPR, R, 1, 1, GROUPED>, k_experts_up<LPR, R, 1, 4, GROUPED>, k_experts_up<LPR, R, 1, 16, GROUPED>)
              : u == 2 ? pick(k_experts_up<LPR, R, 2, 1, GROUPED>, k_experts_up<LPR, R, 2, 4, GROUPED>, k_experts_up<LPR, R, 2, 16, GROUPED>)
              : u == 3 ? pick(k_experts_up<LPR, R, 3, 1, GROUPED>, k_experts_up<LPR, R, 3, 4, GROUPED>, k_experts_up<LPR, R, 3, 16, GROUPED>)
                       : pick(k_experts_up<LPR, R, 5, 1, GROUPED>, k_experts_up<LPR, R, 5, 4, GROUPED>, k_experts_up<LPR, R, 5, 16, GROUPED>);
    const size_t lds = (size_t)k.kp * 4;
    if (lds > 65536) {
        const hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void *>(fn), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
        if (e != hipSuccess) return e;
    }
    hipLaunchKernelGGL(fn, dim3(gemv_grid(k.groups, top), top), dim3(256), lds, s, k);
    return hipGetLastError();
}

template <bool GROUPED>
static hipError_t up_pick(const ExpertsUp &a, hipStream_t s) {
    if (a.cols <= 256) return a.gated ? up_go<16, 2, GROUPED>(a, (a.cols + 127) / 128, s) : up_go<16, 1, GROUPED>(a, (a.cols + 127) / 128, s);
    const int chunks = (a.cols + 511) / 512;
    return a.gated || (long)a.rows * (long)a.r.top >= 4096 ? up_go<64, 2, GROUPED>(a, chunks, s) : up_go<64, 1, GROUPED>(a, chunks, s);
}

hipError_t launch_experts_up(const ExpertsUp &a, hipStream_t s) { return a.r.groups ? up_pick<true>(a, s) : up_pick<false>(a, s); }

template <int LPR, int R>
static hipError_t out_go(const ExpertsOut &a, hipStream_t s) {
    OutK k;
    k.a = a;
    constexpr int CH = LPR * 8;
    k.c0 = (a.cols0 + CH - 1) / CH, k.ce = (a.cols1 + CH - 1) / CH;
    const int chunks = k.c0 + a.top * k.ce, u = chunks >= 8 ? 8 : chunks >= 4 ? 4 : 2;
    k.chunks = (chunks + u - 1) / u * u;
    k.magic = ((1u << 20) + k.ce - 1) / k.ce;
    k.groups = (a.rows + 64 / LPR * R - 1) / (64 / LPR * R);
    const size_t lds = (size_t)k.chunks * CH * 4;
    // (the quotient by multiplication holds while chunks * ce stays below 2^20)
    if (lds > 150 * 1024 || (long)k.chunks * k.ce >= 1 << 20) return hipErrorInvalidValue;
    auto fn = u == 2 ? k_experts_out<LPR, R, 2> : u == 4 ? k_experts_out<LPR, R, 4> : k_experts_out<LPR, R, 8>;
    if (lds > 65536) {
        const hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void *>(fn), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
        if (e != hipSuccess) return e;
    }
    hipLaunchKernelGGL(fn, dim3(gemv_grid(k.groups, 1)), dim3(256), lds, s, k);
    return hipGetLastError();
}

hipError_t launch_experts_out(const ExpertsOut &a, hipStream_t s) {
    auto waste = [&](int ch) { return (double)((a.cols0 + ch - 1) / ch * ch + (long)a.top * ((a.cols1 + ch - 1) / ch * ch)) / (a.cols0 + (double)a.top * a.cols1); };
    auto fits = [&](int ch) { return ((a.cols0 + ch - 1) / ch + (long)a.top * ((a.cols1 + ch - 1) / ch) + 7) / 8 * 8 * ch * 4 <= 150 * 1024; };
    // the longest rows of lanes whose chunks are not padding for the most part (lanes past a row's end load its last columns again: no traffic)
    return waste(512) <= 1.4 * waste(256) && fits(512) ? out_go<64, 1>(a, s) : waste(256) <= 1.3 * waste(128) && fits(256) ? out_go<32, 1>(a, s) : out_go<16, 1>(a, s);
}

}  // namespace bitnet_hip
