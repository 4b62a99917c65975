// kernels_latent.hip -- attention over a latent key / value cache (gfx950).
//
// Per position the cache holds one latent row c [kv_rank] and one rotated key part r [rot_dim] shared by all heads.  A head's
// key is (W_uk c | r) and its value W_uv c.  Two forms:
//   decode  the query is taken into latent space (q' = W_uk^T q) and scores c and r directly; the heads' weighted sums of c go
//           through W_uv afterwards.  k_latent_decode (matrix cores, 16 heads at a time) and k_latent_decode_any (any size, f32 cache).
//   prompt  keys and values of the context are expanded once per layer (matmuls), then k_latent_prefill: flash attention on
//           S^T = K Q^T and O^T = V^T P^T, probabilities staying in registers.
// Scores, running maximum, sum and the weights themselves are f32: a weight enters the matrix cores as a (high, low) pair of
// bf16 values.  A learned sink per head (where there is one) joins the denominator only.
#include "dense.hpp"

namespace bitnet_hip {

// which keys a record covers: whole tiles of kLatentTile keys, `per` tiles per record
__device__ __forceinline__ void split_range(int n_keys, int &per, int &used) {
    const int tiles = (n_keys + kLatentTile - 1) / kLatentTile;
    per = (tiles + kLatentSplits - 1) / kLatentSplits;
    used = (tiles + per - 1) / per;
}

// element i of the rotated part of a query head (raw part at q); elements past 2 * half are zero
template <class T>
__device__ __forceinline__ float rotated(const T *q, const float *cs, const float *sn, int half, int i) {
    const int n = 2 * half, a = min(i, n - 1), b = a < half ? a + half : a - half, c = a < half ? a : a - half;
    const float x = ld_act(q, a), y = ld_act(q, b), s = sn[c], live = i < n ? 1.0f : 0.0f;  // (a product, not a branch around the loads)
    return (x * cs[c] + (a < half ? -y : y) * s) * live;
}

// (no canonicalising v_max of an MFMA result ahead of it; no NaNs here)
__device__ __forceinline__ float max3(float a, float b, float c) {
    float r;
    asm("v_max3_f32 %0, %1, %2, %3" : "=v"(r) : "v"(a), "v"(b), "v"(c));
    return r;
}

size_t latent_scratch_floats(int heads, int ldc, int nq) { return (size_t)nq * heads * kLatentSplits * (kLatentRecHead + ldc); }

// ---- decode, any size -------------------------------------------------------------------------------------------------
// One workgroup per (record, head, query); a wave takes every fourth key, its lanes the latent's columns.
template <class T, int NJ>
__global__ __launch_bounds__(256) void k_latent_decode_any(LatentAttn p) {
    extern __shared__ float vec[];  // [4][ldc]
    __shared__ float sm[4], sl[4];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const int h = blockIdx.y, qi = blockIdx.z;
    const int pos = *p.pos + p.q0 + qi, n_keys = pos + 1;
    int per, used;
    split_range(n_keys, per, used);
    if ((int)blockIdx.x >= used) return;
    const int k0 = blockIdx.x * per * kLatentTile, k1 = min(k0 + per * kLatentTile, n_keys);
    const int half = p.rot_dim / 2;
    const float *qa = p.qabs + ((size_t)qi * p.heads + h) * p.ldc;
    const float *qr = p.q + (size_t)qi * p.ldq + (size_t)h * p.qd + p.dimp;
    constexpr int NR = 4;
    float q[NJ], r[NR], acc[NJ];
#pragma unroll
    for (int j = 0; j < NJ; ++j) {
        const int i = lane + 64 * j;
        q[j] = i < p.ldc ? qa[i] : 0.f;
        acc[j] = 0.f;
    }
#pragma unroll
    for (int j = 0; j < NR; ++j) {
        const int i = lane + 64 * j;
        r[j] = i < p.rot_dim ? rotated(qr, p.rope_cos + (size_t)pos * half, p.rope_sin + (size_t)pos * half, half, i) : 0.f;
    }
    float m = -INFINITY, l = 0.f;
    for (int key = k0 + wave; key < k1; key += 4) {
        const T *c = (const T *)p.ccache + (size_t)key * p.ldc;
        const T *kr = (const T *)p.rcache + (size_t)key * p.ldr;
        float cv[NJ], s = 0.f;
#pragma unroll
        for (int j = 0; j < NJ; ++j) {
            const int i = lane + 64 * j;
            cv[j] = i < p.ldc ? ld_act(c, i) : 0.f;
            s += q[j] * cv[j];
        }
#pragma unroll
        for (int j = 0; j < NR; ++j) {
            const int i = lane + 64 * j;
            if (i < p.rot_dim) s += r[j] * ld_act(kr, i);
        }
        s = wave_sum(s) * p.scale;
        const float mn = fmaxf(m, s), al = expf(m - mn), w = expf(s - mn);
        l = l * al + w;
        m = mn;
#pragma unroll
        for (int j = 0; j < NJ; ++j) acc[j] = acc[j] * al + w * cv[j];
    }
    if (lane == 0) sm[wave] = m, sl[wave] = l;
#pragma unroll
    for (int j = 0; j < NJ; ++j)
        if (lane + 64 * j < p.ldc) vec[wave * p.ldc + lane + 64 * j] = acc[j];
    __syncthreads();
    const float M = fmaxf(fmaxf(sm[0], sm[1]), fmaxf(sm[2], sm[3]));
    float w[4], L = 0.f;
#pragma unroll
    for (int i = 0; i < 4; ++i) {
        w[i] = sm[i] == -INFINITY ? 0.f : expf(sm[i] - M);
        L += w[i] * sl[i];
    }
    float *rec = p.scratch + (((size_t)qi * p.heads + h) * kLatentSplits + blockIdx.x) * (kLatentRecHead + p.ldc);
    for (int i = tid; i < p.ldc; i += 256)
        rec[kLatentRecHead + i] = (w[0] * vec[i] + w[1] * vec[p.ldc + i]) + (w[2] * vec[2 * p.ldc + i] + w[3] * vec[3 * p.ldc + i]);
    if (tid == 0) rec[0] = M, rec[1] = L;
}

// ---- decode, matrix cores ---------------------------------------------------------------------------------------------
// One workgroup per (record, 16 heads, query), 64 keys per step, eight waves.  Scores: wave w takes keys [16 (w & 3), + 16) and one half
// of the columns, the rows going from memory straight into the MFMA's B operand (a lane: one key, eight columns); the f32 query is a
// (high, low) pair.  The same registers leave the tile transposed in LDS (key pairs from two neighbouring lanes), and the waves share
// the columns of O += P C.
constexpr int kDecKK = 20;  // most 32-column steps of ldc + ldr
constexpr int kDecNT = 5;   // most 16-column tiles of ldc per wave
constexpr int kCtStride = kLatentTile * 2 + 16;

// NCK, NRK: 32-column steps of the latent and of the rotated part when known at compile time (no branches between the loads), else 0
template <int NCK, int NRK>
__global__ __launch_bounds__(512) void k_latent_decode(LatentAttn p) {
    extern __shared__ __attribute__((aligned(16))) uint8_t lds[];
    __shared__ float smax[4][16], ssum[4][16];
    __shared__ f32x4 spart[4][64];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, r16 = lane & 15, g = lane >> 4;
    const int kg = wave & 3, half_cols = wave >> 2;
    const int h0 = blockIdx.y * 16, qi = blockIdx.z;
    constexpr int MKK = NCK ? (NCK + NRK + 1) / 2 : kDecKK / 2, MNT = NCK ? NCK / 4 : kDecNT;
    const int nck = NCK ? NCK : p.ldc / 32, nkk = NCK ? NCK + NRK : nck + p.ldr / 32, kt = nkk * 32, ntiles = nck * 2, ldc = nck * 32;
    const int kk0 = half_cols * ((nkk + 1) / 2), kn = half_cols ? nkk / 2 : (nkk + 1) / 2;  // this wave's steps
    const int qs = kt * 2 + 16;  // bytes per query row
    uint8_t *ct = lds, *qh = ct + (size_t)ldc * kCtStride, *ql = qh + 16 * qs, *ph = ql + 16 * qs, *pl = ph + 16 * kCtStride;
    const uint16_t *C = (const uint16_t *)p.ccache, *R = (const uint16_t *)p.rcache;
    u32x4 b[MKK];
    auto fetch = [&](int key0) {
        const int key = key0 + kg * 16 + r16;  // below the capacity, a multiple of 64
#pragma unroll
        for (int i = 0; i < MKK; ++i) {
            const int kk = min(kk0 + i, nkk - 1);
            const uint16_t *src = kk < nck ? C + (size_t)key * ldc + kk * 32 : R + (size_t)key * p.ldr + (kk - nck) * 32;
            b[i] = *reinterpret_cast<const u32x4 *>(src + g * 8);
        }
    };
    // up to kLatentSplits tiles a record is one tile: requested before the position is known (any tile below the capacity may be read)
    fetch(blockIdx.x * kLatentTile);
    const int pos = *p.pos + p.q0 + qi, n_keys = pos + 1;
    int per, used;
    split_range(n_keys, per, used);
    if ((int)blockIdx.x >= used) return;
    const int k0 = blockIdx.x * per * kLatentTile, k1 = min(k0 + per * kLatentTile, n_keys);
    if (per > 1) fetch(k0);
    {
        // the query rows, 32 threads each: latent part, then the rotated part
        const int half = p.rot_dim / 2, row = tid >> 5, c4 = (tid & 31) * 4, h = min(h0 + row, p.heads - 1);
        const float *qa = p.qabs + ((size_t)qi * p.heads + h) * ldc;
        const float *qr = p.q + (size_t)qi * p.ldq + (size_t)h * p.qd + p.dimp;
        const float *cs = p.rope_cos + (size_t)pos * half, *sn = p.rope_sin + (size_t)pos * half;
        constexpr int NQ = NCK ? (NCK + 3) / 4 : kDecNT;  // 128 columns at a time
        f32x4 v[NQ];
#pragma unroll
        for (int t = 0; t < NQ; ++t) v[t] = *reinterpret_cast<const f32x4 *>(qa + min(t * 128 + c4, ldc - 4));
        auto put = [&](int i, float x, float y) {
            uint32_t hi, lo;
            split2(x, y, hi, lo);
            *reinterpret_cast<uint32_t *>(qh + row * qs + i * 2) = hi;
            *reinterpret_cast<uint32_t *>(ql + row * qs + i * 2) = lo;
        };
        for (int i = (tid & 31) * 2; i < p.ldr; i += 64) put(ldc + i, rotated(qr, cs, sn, half, i), rotated(qr, cs, sn, half, i + 1));
#pragma unroll
        for (int t = 0; t < NQ; ++t)
            if (t * 128 + c4 < ldc) {
                put(t * 128 + c4, v[t].x, v[t].y);
                put(t * 128 + c4 + 2, v[t].z, v[t].w);
            }
    }
    __syncthreads();
    f32x4 o[MNT];
#pragma unroll
    for (int t = 0; t < MNT; ++t) o[t] = f32x4{0.f, 0.f, 0.f, 0.f};
    float m[4], l[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) m[i] = -INFINITY, l[i] = 0.f;
    const bool even = (lane & 1) == 0;
    for (int key0 = k0; key0 < k1; key0 += kLatentTile) {
        f32x4 s4[4];  // independent chains: high / low half of the query, even / odd step
#pragma unroll
        for (int i = 0; i < 4; ++i) s4[i] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int i = 0; i < MKK; ++i) {
            if (i >= kn) continue;
            const int kk = kk0 + i;
            const bf16x8 bv = __builtin_bit_cast(bf16x8, b[i]);
            s4[i & 1] = mfma_bf16(*reinterpret_cast<const bf16x8 *>(qh + r16 * qs + kk * 64 + g * 16), bv, s4[i & 1]);
            s4[2 + (i & 1)] = mfma_bf16(*reinterpret_cast<const bf16x8 *>(ql + r16 * qs + kk * 64 + g * 16), bv, s4[2 + (i & 1)]);
            if (kk < nck) {
                const uint32_t x0 = even ? b[i].z : b[i].x, x1 = even ? b[i].w : b[i].y;
                const uint32_t a0 = even ? b[i].x : b[i].z, a1 = even ? b[i].y : b[i].w;
                const uint32_t r0 = (uint32_t)__builtin_amdgcn_update_dpp(0, (int)x0, 0xb1, 0xf, 0xf, true);
                const uint32_t r1 = (uint32_t)__builtin_amdgcn_update_dpp(0, (int)x1, 0xb1, 0xf, 0xf, true);
                const uint32_t f0 = even ? a0 : r0, s0 = even ? r0 : a0, f1 = even ? a1 : r1, s1 = even ? r1 : a1;
                uint8_t *dst = ct + (size_t)(kk * 32 + g * 8 + (even ? 0 : 4)) * kCtStride + (kg * 16 + (r16 & ~1)) * 2;
                *reinterpret_cast<uint32_t *>(dst) = __builtin_amdgcn_perm(s0, f0, 0x05040100u);
                *reinterpret_cast<uint32_t *>(dst + kCtStride) = __builtin_amdgcn_perm(s0, f0, 0x07060302u);
                *reinterpret_cast<uint32_t *>(dst + 2 * kCtStride) = __builtin_amdgcn_perm(s1, f1, 0x05040100u);
                *reinterpret_cast<uint32_t *>(dst + 3 * kCtStride) = __builtin_amdgcn_perm(s1, f1, 0x07060302u);
            }
        }
        if (key0 + kLatentTile < k1) fetch(key0 + kLatentTile);
        f32x4 s = (s4[0] + s4[1]) + (s4[2] + s4[3]);
        if (half_cols) spart[kg][lane] = s;
        __syncthreads();
        if (!half_cols) {
            s += spart[kg][lane];
            const bool live = key0 + kg * 16 + r16 < k1;
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                s[i] = live ? s[i] * p.scale : -INFINITY;
                const float mx = row_max(s[i]);
                if (r16 == 0) smax[kg][g * 4 + i] = mx;
            }
        }
        __syncthreads();
        float al[4];
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            const int row = g * 4 + i;
            const float mn = fmaxf(m[i], fmaxf(fmaxf(smax[0][row], smax[1][row]), fmaxf(smax[2][row], smax[3][row])));
            al[i] = expf(m[i] - mn);
            m[i] = mn;
        }
        if (!half_cols)
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                const int row = g * 4 + i;
                const float w = expf(s[i] - m[i]);
                l[i] = l[i] * al[i] + row_sum(w);
                uint32_t hi, lo;
                split2(w, 0.f, hi, lo);
                *reinterpret_cast<uint16_t *>(ph + row * kCtStride + (kg * 16 + r16) * 2) = (uint16_t)hi;
                *reinterpret_cast<uint16_t *>(pl + row * kCtStride + (kg * 16 + r16) * 2) = (uint16_t)lo;
            }
        __syncthreads();
        bf16x8 pa[2][2];
#pragma unroll
        for (int ks = 0; ks < 2; ++ks) {
            pa[ks][0] = *reinterpret_cast<const bf16x8 *>(ph + r16 * kCtStride + ks * 64 + g * 16);
            pa[ks][1] = *reinterpret_cast<const bf16x8 *>(pl + r16 * kCtStride + ks * 64 + g * 16);
        }
#pragma unroll
        for (int t = 0; t < MNT; ++t) {
            const int tile = t * 8 + wave;
            if (tile >= ntiles) continue;
            o[t] *= f32x4{al[0], al[1], al[2], al[3]};
#pragma unroll
            for (int ks = 0; ks < 2; ++ks) {
                const bf16x8 cv = *reinterpret_cast<const bf16x8 *>(ct + (size_t)(tile * 16 + r16) * kCtStride + ks * 64 + g * 16);
                o[t] = mfma_bf16(pa[ks][0], cv, o[t]);
                o[t] = mfma_bf16(pa[ks][1], cv, o[t]);
            }
        }
        __syncthreads();
    }
    if (!half_cols && r16 == 0)
#pragma unroll
        for (int i = 0; i < 4; ++i) ssum[kg][g * 4 + i] = l[i];
    __syncthreads();
#pragma unroll
    for (int i = 0; i < 4; ++i) {
        const int row = g * 4 + i, h = h0 + row;
        if (h >= p.heads) continue;
        float *rec = p.scratch + (((size_t)qi * p.heads + h) * kLatentSplits + blockIdx.x) * (kLatentRecHead + ldc);
#pragma unroll
        for (int t = 0; t < MNT; ++t)
            if (t * 8 + wave < ntiles) rec[kLatentRecHead + (t * 8 + wave) * 16 + r16] = o[t][i];
        if (wave == 0 && r16 == 0) rec[0] = m[i], rec[1] = (ssum[0][row] + ssum[1][row]) + (ssum[2][row] + ssum[3][row]);
    }
}

template <class T>
static hipError_t decode_any(const LatentAttn &a, dim3 grid, hipStream_t s) {
    const size_t lds = (size_t)4 * a.ldc * sizeof(float);
    const int nj = (a.ldc + 63) / 64;
    if (a.rot_dim > 256 || nj > 16) return hipErrorInvalidValue;
    if (nj <= 1)
        hipLaunchKernelGGL((k_latent_decode_any<T, 1>), grid, dim3(256), lds, s, a);
    else if (nj <= 4)
        hipLaunchKernelGGL((k_latent_decode_any<T, 4>), grid, dim3(256), lds, s, a);
    else if (nj <= 8)
        hipLaunchKernelGGL((k_latent_decode_any<T, 8>), grid, dim3(256), lds, s, a);
    else
        hipLaunchKernelGGL((k_latent_decode_any<T, 16>), grid, dim3(256), lds, s, a);
    return hipGetLastError();
}

hipError_t launch_latent_decode(const LatentAttn &a, hipStream_t s) {
    const int splits = min(kLatentSplits, (a.capacity + kLatentTile - 1) / kLatentTile);
    if (a.f32) return decode_any<float>(a, dim3(splits, a.heads, a.nq), s);
    const int kt = a.ldc + a.ldr;
    if (kt > 32 * kDecKK || a.ldc > 128 * kDecNT || a.ldc % 64 || a.ldr % 32) return decode_any<uint16_t>(a, dim3(splits, a.heads, a.nq), s);
    const size_t lds = (size_t)a.ldc * kCtStride + (size_t)32 * (kt * 2 + 16) + (size_t)32 * kCtStride;
    auto fn = a.ldc == 512 && a.ldr == 64 ? k_latent_decode<16, 2> : k_latent_decode<0, 0>;
    if (lds > 65536) {
        const hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void *>(fn), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
        if (e != hipSuccess) return e;
    }
    hipLaunchKernelGGL(fn, dim3(splits, (a.heads + 15) / 16, a.nq), dim3(512), lds, s, a);
    return hipGetLastError();
}

// ---- the records of a head -> its value vector --------------------------------------------------------------------------
// Every workgroup merges the head's records (running maxima, sums, the sink) in LDS and takes a share of W_uv's rows.
template <class TO>
__global__ __launch_bounds__(512) void k_latent_merge(LatentMerge p) {
    extern __shared__ __attribute__((aligned(16))) float o[];  // [ldc], then four partial vectors
    static_assert(kLatentSplits == 128, "two records per lane of a wave");
    __shared__ float ws[kLatentSplits], sden;
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const int h = blockIdx.x, qi = blockIdx.z;
    int per, used;
    split_range(*p.pos + p.q0 + qi + 1, per, used);
    const size_t stride = kLatentRecHead + p.ldc;
    const float *rec = p.scratch + ((size_t)qi * p.heads + h) * kLatentSplits * stride;
    if (wave == 0) {
        const float sink = p.sink ? p.sink[h] : -INFINITY;
        float mv[2], lv[2], M = sink;
#pragma unroll
        for (int e = 0; e < 2; ++e) {
            const int r = lane + 64 * e;
            mv[e] = r < used ? rec[r * stride] : -INFINITY;
            lv[e] = r < used ? rec[r * stride + 1] : 0.f;
            M = fmaxf(M, mv[e]);
        }
        M = rows_max(row_max(M));
        float den = 0.f;
#pragma unroll
        for (int e = 0; e < 2; ++e) {
            const float w = lane + 64 * e < used ? expf(mv[e] - M) : 0.f;
            ws[lane + 64 * e] = w;
            den += w * lv[e];
        }
        den = wave_sum(den) + expf(sink - M);
        if (lane == 0) sden = den;
    }
    __syncthreads();
    float *part = o + p.ldc;
    const int grp = tid >> 7, t = tid & 127;
    for (int i = t * 4; i < p.ldc; i += 512) {
        f32x4 a = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll 16
        for (int r = grp; r < used; r += 4) a += ws[r] * *reinterpret_cast<const f32x4 *>(rec + r * stride + kLatentRecHead + i);
        *reinterpret_cast<f32x4 *>(part + grp * p.ldc + i) = a;
    }
    __syncthreads();
    const float inv = 1.0f / sden;
    for (int i = tid; i < p.ldc; i += 512) o[i] = ((part[i] + part[p.ldc + i]) + (part[2 * p.ldc + i] + part[3 * p.ldc + i])) * inv;
    __syncthreads();
    const int share = (p.vdimp + gridDim.y - 1) / gridDim.y, v0 = blockIdx.y * share, v1 = min(v0 + share, p.vdimp);
    TO *out = (TO *)p.out + (size_t)qi * p.ldo + (size_t)h * p.vdimp;
    for (int v = v0 + wave; v < v1; v += 8) {
        const uint16_t *w = p.uv + ((size_t)h * p.vdimp + v) * p.ldc;
        float acc = 0.f;
        for (int i = lane * 8; i < p.ldc; i += 512) {
            const u32x4 wv = *reinterpret_cast<const u32x4 *>(w + i);
            const f32x4 x0 = *reinterpret_cast<const f32x4 *>(o + i), x1 = *reinterpret_cast<const f32x4 *>(o + i + 4);
            acc = fmaf(x0.x, bf2f(wv.x & 0xffffu), fmaf(x0.y, bf2f(wv.x >> 16), acc));
            acc = fmaf(x0.z, bf2f(wv.y & 0xffffu), fmaf(x0.w, bf2f(wv.y >> 16), acc));
            acc = fmaf(x1.x, bf2f(wv.z & 0xffffu), fmaf(x1.y, bf2f(wv.z >> 16), acc));
            acc = fmaf(x1.z, bf2f(wv.w & 0xffffu), fmaf(x1.w, bf2f(wv.w >> 16), acc));
        }
        acc = wave_sum(acc);
        if (lane == 0) st_act(out, v, acc);
    }
}

hipError_t launch_latent_merge(const LatentMerge &a, hipStream_t s) {
    const int shares = a.nq > 1 ? 1 : (a.vdimp >= 64 ? 4 : 1);
    const size_t lds = (size_t)5 * a.ldc * sizeof(float);
    if (lds > 65536) return hipErrorInvalidValue;
    if (a.out_bf16)
        hipLaunchKernelGGL(k_latent_merge<uint16_t>, dim3(a.heads, shares, a.nq), dim3(512), lds, s, a);
    else
        hipLaunchKernelGGL(k_latent_merge<float>, dim3(a.heads, shares, a.nq), dim3(512), lds, s, a);
    return hipGetLastError();
}

// ---- prompt -----------------------------------------------------------------------------------------------------------
// One workgroup: one head, 64 QT queries, four waves of 16 QT; key tiles of 64 staged through registers into LDS one step ahead.
// NK: 32-column steps of a key (dimp + ldr), NV: 16-row tiles of V^T.
template <int NK, int NV, int QT>
__global__ __launch_bounds__(256, NV > 8 ? 1 : QT == 1 ? 3 : 2) void k_latent_prefill(LatentAttn p, int n_qb) {
    extern __shared__ __attribute__((aligned(16))) uint8_t lds[];
    constexpr int KS = NK * 64 + 16, VS = kLatentTile * 2 + 16, NVL = NV / 2;
    uint8_t *lk = lds, *lv = lds + kLatentTile * KS;
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, r16 = lane & 15, g = lane >> 4;
    // Consecutive workgroups go to the eight XCDs in turn.  Longest blocks first; an XCD keeps heads / 8 heads of its own (their keys
    // and values stay in its L2), the heads left over move from XCD to XCD with the block so that all eight carry the same work.
    const int x = blockIdx.x & 7, rest = blockIdx.x >> 3, own = p.heads >> 3, left = p.heads & 7, per = own + (left ? 1 : 0);
    const int level = rest / per, slot = rest - level * per, r = (x + 8 * left - (level % 8) * left) & 7;
    if (slot == own && r >= left) return;
    const int h = slot < own ? x * own + slot : 8 * own + r, qb = n_qb - 1 - level;
    const int q0 = qb * 64 * QT, pos0 = p.n_ctx - p.nq;
    const int qw = q0 + wave * 16 * QT;  // this wave's first query
    const int half = p.rot_dim / 2;
    bf16x8 qf[QT][NK];
    int qpos[QT];
#pragma unroll
    for (int t = 0; t < QT; ++t) {
        const int qi = min(qw + t * 16 + r16, p.nq - 1);
        qpos[t] = pos0 + qw + t * 16 + r16;
        const float sign = p.scale < 0.f ? -1.0f : 1.0f;
        const uint16_t *q = (const uint16_t *)p.qb + (size_t)qi * p.ldq + (size_t)h * p.qd;
        const float *cs = p.rope_cos + (size_t)(pos0 + qi) * half, *sn = p.rope_sin + (size_t)(pos0 + qi) * half;
#pragma unroll
        for (int kk = 0; kk < NK; ++kk) {
            const int d = kk * 32 + g * 8;
            if (kk * 32 < p.dimp) {
                qf[t][kk] = *reinterpret_cast<const bf16x8 *>(q + d);
                if (p.scale < 0.f)
#pragma unroll
                    for (int e = 0; e < 8; ++e) qf[t][kk][e] = -qf[t][kk][e];
            } else {
#pragma unroll
                for (int e = 0; e < 8; ++e) qf[t][kk][e] = (__bf16)(sign * rotated(q + p.dimp, cs, sn, half, d + e - p.dimp));
            }
        }
    }
    // scores stay unscaled up to the exponential (their maximum is then the maximum of the scaled ones: a negative scale's sign goes
    // into the query)
    const float c2 = fabsf(p.scale) * 1.44269504088896f, sink2 = p.sink ? p.sink[h] * 1.44269504088896f : -1e30f;  // (every query sees the first tile's first key)
    f32x4 o[NV][QT];
    float m[QT], l[QT];
#pragma unroll
    for (int t = 0; t < QT; ++t) {
        m[t] = sink2;
        l[t] = p.sink && g == 0 ? 1.0f : 0.0f;
#pragma unroll
        for (int v = 0; v < NV; ++v) o[v][t] = f32x4{0.f, 0.f, 0.f, 0.f};
    }
    const uint16_t *K = (const uint16_t *)p.k + (size_t)h * p.dimp, *R = (const uint16_t *)p.rcache;
    const uint16_t *V = (const uint16_t *)p.vt + (size_t)h * p.vdimp * p.ldvt;
    const size_t ldk = (size_t)p.heads * p.dimp;
    u32x4 kreg[NK], vreg[NVL];
    // four threads per key: 64 bytes of every 32-column step, latent keys first, then the shared rotated part (both multiples of 32
    // columns: one address form per step); eight threads per row of V^T
    const unsigned koff = (unsigned)((tid >> 2) * ldk * 2 + (tid & 3) * 16), roff = (unsigned)((tid >> 2) * p.ldr * 2 + (tid & 3) * 16);
    const unsigned voff = (unsigned)((tid >> 3) * p.ldvt * 2 + (tid & 7) * 16);
    auto fetch = [&](int key0) {
        const char *kb = (const char *)(K + (size_t)key0 * ldk), *rb = (const char *)(R + (size_t)key0 * p.ldr), *vb = (const char *)(V + key0);
#pragma unroll
        for (int j = 0; j < NK; ++j) {
            if (j * 32 < p.dimp)
                kreg[j] = *reinterpret_cast<const u32x4 *>(kb + j * 64 + koff);
            else if (j * 32 < p.qd)
                kreg[j] = *reinterpret_cast<const u32x4 *>(rb + (j * 64 - p.dimp * 2) + roff);
        }
#pragma unroll
        for (int j = 0; j < NVL; ++j)
            if (j * 32 < p.vdimp) vreg[j] = *reinterpret_cast<const u32x4 *>(vb + (size_t)j * 64 * p.ldvt + voff);
    };
#pragma unroll
    for (int j = 0; j < NK; ++j) kreg[j] = u32x4{0u, 0u, 0u, 0u};
#pragma unroll
    for (int j = 0; j < NVL; ++j) vreg[j] = u32x4{0u, 0u, 0u, 0u};
    const int n_tiles = (min(p.n_ctx, pos0 + q0 + 64 * QT) + kLatentTile - 1) / kLatentTile;
    fetch(0);
    for (int kt0 = 0; kt0 < n_tiles; ++kt0) {
        const int key0 = kt0 * kLatentTile;
        __syncthreads();
#pragma unroll
        for (int j = 0; j < NK; ++j) *reinterpret_cast<u32x4 *>(lk + (tid >> 2) * KS + j * 64 + (tid & 3) * 16) = kreg[j];
#pragma unroll
        for (int j = 0; j < NVL; ++j) *reinterpret_cast<u32x4 *>(lv + ((tid >> 3) + 32 * j) * VS + (tid & 7) * 16) = vreg[j];
        __syncthreads();
        if (kt0 + 1 < n_tiles) fetch(key0 + kLatentTile);
        if (key0 > pos0 + qw + 16 * QT - 1) continue;  // every key of the tile lies ahead of this wave's queries
        f32x4 s[4][QT];
#pragma unroll
        for (int kt = 0; kt < 4; ++kt) {
#pragma unroll
            for (int t = 0; t < QT; ++t) s[kt][t] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int kk = 0; kk < NK; ++kk) {
                const bf16x8 a = *reinterpret_cast<const bf16x8 *>(lk + (kt * 16 + r16) * KS + kk * 64 + g * 16);
#pragma unroll
                for (int t = 0; t < QT; ++t) s[kt][t] = mfma_bf16(a, qf[t][kk], s[kt][t]);
            }
        }
        if (key0 + kLatentTile - 1 > pos0 + qw)  // the diagonal
#pragma unroll
            for (int t = 0; t < QT; ++t)
#pragma unroll
                for (int kt = 0; kt < 4; ++kt)
#pragma unroll
                    for (int i = 0; i < 4; ++i) s[kt][t][i] = key0 + kt * 16 + g * 4 + i > qpos[t] ? -INFINITY : s[kt][t][i];
        float mn[QT];
        bool grows = false;
#pragma unroll
        for (int t = 0; t < QT; ++t) {
            // (hipcc does not count the wait states between an MFMA's result and inline asm that reads it)
            asm volatile("s_nop 11" : "+v"(s[0][t]), "+v"(s[1][t]), "+v"(s[2][t]), "+v"(s[3][t]));
            float mx = max3(s[0][t][0], s[0][t][1], s[0][t][2]);
            mx = max3(mx, s[0][t][3], s[1][t][0]);
            mx = max3(mx, s[1][t][1], s[1][t][2]);
            mx = max3(mx, s[1][t][3], s[2][t][0]);
            mx = max3(mx, s[2][t][1], s[2][t][2]);
            mx = max3(mx, s[2][t][3], s[3][t][0]);
            mx = max3(mx, s[3][t][1], s[3][t][2]);
            mx = rows_max(max3(mx, s[3][t][3], -INFINITY));
            mn[t] = fmaxf(m[t], mx * c2);
            grows = grows || mn[t] > m[t];
        }
        if (__any(grows)) {
#pragma unroll
            for (int t = 0; t < QT; ++t) {
                const float al = __builtin_amdgcn_exp2f(m[t] - mn[t]);
                m[t] = mn[t];
                l[t] *= al;
#pragma unroll
                for (int v = 0; v < NV; ++v) o[v][t] *= al;
            }
        }
        bf16x8 ph[2][QT], pl[2][QT];
#pragma unroll
        for (int ks = 0; ks < 2; ++ks)
#pragma unroll
            for (int t = 0; t < QT; ++t) {
                u32x4 hi, lo;
#pragma unroll
                for (int j = 0; j < 4; ++j) {
                    const int kt = 2 * ks + (j >> 1), i = (j & 1) * 2;
                    const float a = __builtin_amdgcn_exp2f(fmaf(s[kt][t][i], c2, -m[t])), b = __builtin_amdgcn_exp2f(fmaf(s[kt][t][i + 1], c2, -m[t]));
                    l[t] += a + b;
                    uint32_t uh, ul;
                    split2(a, b, uh, ul);
                    hi[j] = uh;
                    lo[j] = ul;
                }
                ph[ks][t] = __builtin_bit_cast(bf16x8, hi);
                pl[ks][t] = __builtin_bit_cast(bf16x8, lo);
            }
#pragma unroll
        for (int v = 0; v < NV; ++v)
#pragma unroll
            for (int ks = 0; ks < 2; ++ks) {
                const uint8_t *row = lv + (v * 16 + r16) * VS + ks * 64 + g * 8;
                const u32x2 a0 = *reinterpret_cast<const u32x2 *>(row), a1 = *reinterpret_cast<const u32x2 *>(row + 32);
                const bf16x8 a = __builtin_bit_cast(bf16x8, u32x4{a0.x, a0.y, a1.x, a1.y});
#pragma unroll
                for (int t = 0; t < QT; ++t) {
                    o[v][t] = mfma_bf16(a, ph[ks][t], o[v][t]);
                    o[v][t] = mfma_bf16(a, pl[ks][t], o[v][t]);
                }
            }
    }
#pragma unroll
    for (int t = 0; t < QT; ++t) {
        const int qi = qw + t * 16 + r16;
        const float inv = 1.0f / rows_sum(l[t]);
        if (qi >= p.nq) continue;
        uint16_t *dst = (uint16_t *)p.out + (size_t)qi * p.ldo + (size_t)h * p.vdimp + g * 4;
#pragma unroll
        for (int v = 0; v < NV; ++v)
            if (v * 16 < p.vdimp) {
                const f32x4 r = o[v][t] * inv;
                *reinterpret_cast<bf16x4 *>(dst + v * 16) = bf16x4{(__bf16)r.x, (__bf16)r.y, (__bf16)r.z, (__bf16)r.w};
            }
    }
}

bool latent_prefill_supported(int qd, int vdimp) { return qd <= 256 && vdimp <= 256; }

template <int NK, int NV, int QT>
static hipError_t prefill_go(const LatentAttn &a, hipStream_t s) {
    const int n_qb = (a.nq + 64 * QT - 1) / (64 * QT);
    const size_t lds = (size_t)kLatentTile * (NK * 64 + 16) + (size_t)NV * 16 * (kLatentTile * 2 + 16);
    if (lds > 65536) {
        const hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void *>(k_latent_prefill<NK, NV, QT>), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
        if (e != hipSuccess) return e;
    }
    hipLaunchKernelGGL((k_latent_prefill<NK, NV, QT>), dim3(8 * ((a.heads + 7) / 8) * n_qb), dim3(256), lds, s, a, n_qb);
    return hipGetLastError();
}

hipError_t launch_latent_prefill(const LatentAttn &a, hipStream_t s) {
    const int nk = a.qd / 32, nv = a.vdimp / 16;
    if (a.qd % 32 || a.dimp % 32 || a.vdimp % 32 || !latent_prefill_supported(a.qd, a.vdimp)) return hipErrorInvalidValue;
    if (nv > 8) return prefill_go<8, 16, 1>(a, s);
    if (nk <= 2) return nv <= 2 ? prefill_go<2, 2, 2>(a, s) : nv <= 4 ? prefill_go<2, 4, 2>(a, s) : prefill_go<2, 8, 2>(a, s);
    if (nk <= 4) return nv <= 4 ? prefill_go<4, 4, 2>(a, s) : prefill_go<4, 8, 2>(a, s);
    if (nk <= 6) return prefill_go<6, 8, 2>(a, s);
    return prefill_go<8, 8, 2>(a, s);
}

}  // namespace bitnet_hip
