// kernels_linear.hip -- linear attention with a constant decay per head (gfx950):
//   S_t = d S_(t-1) + k_t v_t^T,  o_t = S_t^T q_t,  S in f32, carried from call to call.
// The state is kept transposed, [head][value][key].
//   k_linear_recurrent  token by token (the decode step; f32 inputs)
//   the chunked form    blocks of kLinBlock tokens: k_linear_sums (each block's own contribution), k_linear_scan (the state ahead
//                       of every block, f32), k_linear_out (state part + the causal part inside the block) on the matrix cores.
// In the chunked form f32 operands (decayed keys, decayed scores, states) enter the matrix cores as (high, low) bf16 pairs.
// Powers of the decay come from a table the host computed in double precision.
#include "dense.hpp"

namespace bitnet_hip {

// ---- token by token ---------------------------------------------------------------------------------------------------
// a wave: RV value rows, its lanes the keys' columns
template <int NJ, int RV>
__global__ __launch_bounds__(256) void k_linear_recurrent(LinearAttn p) {
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, h = blockIdx.y;
    const int v0 = (blockIdx.x * 4 + wave) * RV;
    if (v0 >= p.vdimp) return;
    const float d = p.decay_pow[(size_t)h * (kLinBlock + 1) + 1];
    float s[RV][NJ];
    float *st = p.state + ((size_t)h * p.vdimp + v0) * p.dimp;
#pragma unroll
    for (int r = 0; r < RV; ++r)
#pragma unroll
        for (int j = 0; j < NJ; ++j) s[r][j] = lane + 64 * j < p.dimp ? st[(size_t)r * p.dimp + lane + 64 * j] : 0.f;
    for (int t = 0; t < p.n; ++t) {
        const float *row = (const float *)p.qkv + (size_t)t * p.ld;
        const float *q = row + (size_t)h * p.dimp, *k = q + (size_t)p.heads * p.dimp;
        const float *v = row + 2 * (size_t)p.heads * p.dimp + (size_t)h * p.vdimp + v0;
        float qv[NJ], kv[NJ], o[RV];
#pragma unroll
        for (int j = 0; j < NJ; ++j) {
            const bool ok = lane + 64 * j < p.dimp;
            qv[j] = ok ? q[lane + 64 * j] : 0.f;
            kv[j] = ok ? k[lane + 64 * j] : 0.f;
        }
#pragma unroll
        for (int r = 0; r < RV; ++r) {
            const float vr = v[r];
            o[r] = 0.f;
#pragma unroll
            for (int j = 0; j < NJ; ++j) {
                s[r][j] = d * s[r][j] + kv[j] * vr;
                o[r] += s[r][j] * qv[j];
            }
            o[r] = wave_sum(o[r]);
        }
        if (lane == 0)
#pragma unroll
            for (int r = 0; r < RV; ++r) p.out[(size_t)t * p.ldo + (size_t)h * p.vdimp + v0 + r] = o[r];
    }
#pragma unroll
    for (int r = 0; r < RV; ++r)
#pragma unroll
        for (int j = 0; j < NJ; ++j)
            if (lane + 64 * j < p.dimp) st[(size_t)r * p.dimp + lane + 64 * j] = s[r][j];
}

hipError_t launch_linear_recurrent(const LinearAttn &a, hipStream_t s) {
    constexpr int RV = 4;  // vdimp is a multiple of 16
    if (a.vdimp % 16) return hipErrorInvalidValue;
    const dim3 grid(a.vdimp / (4 * RV), a.heads);
    const int nj = (a.dimp + 63) / 64;
    if (nj <= 1)
        hipLaunchKernelGGL((k_linear_recurrent<1, RV>), grid, dim3(256), 0, s, a);
    else if (nj <= 2)
        hipLaunchKernelGGL((k_linear_recurrent<2, RV>), grid, dim3(256), 0, s, a);
    else if (nj <= 4)
        hipLaunchKernelGGL((k_linear_recurrent<4, RV>), grid, dim3(256), 0, s, a);
    else if (nj <= 8)
        hipLaunchKernelGGL((k_linear_recurrent<8, RV>), grid, dim3(256), 0, s, a);
    else
        return hipErrorInvalidValue;
    return hipGetLastError();
}

// ---- chunked ----------------------------------------------------------------------------------------------------------
struct LinearWs {
    float *sums;          // [head][block][vdimp][dimp]
    uint16_t *hi, *lo;    // the state ahead of each block, same shape
    int nb;
};

// A transposed [column][token] tile in LDS: 256 bytes per column, its sixteen 16-byte units (eight tokens each) permuted per column so
// that both the pair-wise writes (eight column groups at once) and the fragment reads (sixteen columns at once) cover all 64 banks.
static_assert(kLinBlock == 128, "the tile's permutation is made for 128 tokens");
constexpr int kTileBytes = kLinBlock * 2;
__device__ __forceinline__ int tile_at(int col, int token) {
    const int c = col >> 3, f = (2 * ((col ^ c) & 7)) ^ (c & 1);
    return col * kTileBytes + ((((token >> 3) ^ f) & 15) << 4) + (token & 7) * 2;
}

// 16 bytes of row t at column c with both clamped into the matrix (loads stay unconditional), and their clearing outside of it
__device__ __forceinline__ u32x4 load_at(const uint16_t *m, size_t ld, int t, int n, int c, int cols) {
    return *reinterpret_cast<const u32x4 *>(m + (size_t)min(t, n - 1) * ld + min(c, cols - 8));
}
__device__ __forceinline__ u32x4 zero_outside(u32x4 v, int t, int n, int c, int cols) {
    const uint32_t keep = t < n && c < cols ? 0xffffffffu : 0u;
    return u32x4{v.x & keep, v.y & keep, v.z & keep, v.w & keep};
}

// two tokens' eight columns -> eight (token, token + 1) dwords
__device__ __forceinline__ void pair_columns(u32x4 a, u32x4 b, uint32_t out[8]) {
#pragma unroll
    for (int i = 0; i < 4; ++i) {
        out[2 * i] = __builtin_amdgcn_perm(b[i], a[i], 0x05040100u);
        out[2 * i + 1] = __builtin_amdgcn_perm(b[i], a[i], 0x07060302u);
    }
}

// sums[block] = sum over the block's tokens t of d^(last - t) v_t k_t^T, one 64 x 64 piece per workgroup
__global__ __launch_bounds__(256) void k_linear_sums(LinearAttn p, LinearWs w) {
    extern __shared__ __attribute__((aligned(16))) uint8_t lds[];
    uint8_t *lv = lds, *kh = lds + 64 * kTileBytes, *kl = kh + 64 * kTileBytes;
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, r16 = lane & 15, g = lane >> 4;
    const int blk = blockIdx.x, h = blockIdx.y, nk = (p.dimp + 63) / 64;
    const int k0 = (blockIdx.z % nk) * 64, v0 = (blockIdx.z / nk) * 64;
    const int t0 = blk * kLinBlock, len = min(kLinBlock, p.n - t0);
    const float *pw = p.decay_pow + (size_t)h * (kLinBlock + 1);
    const uint16_t *K = (const uint16_t *)p.qkv + (size_t)(p.heads + h) * p.dimp, *V = (const uint16_t *)p.qkv + 2 * (size_t)p.heads * p.dimp + (size_t)h * p.vdimp;
    K += (size_t)t0 * p.ld, V += (size_t)t0 * p.ld;
    u32x4 kv[2][4];
#pragma unroll
    for (int j = 0; j < 2; ++j) {
        const int idx = tid + 256 * j, c = (idx & 7) * 8, t = (idx >> 3) * 2;
        kv[j][0] = load_at(V, p.ld, t, len, v0 + c, p.vdimp);
        kv[j][1] = load_at(V, p.ld, t + 1, len, v0 + c, p.vdimp);
        kv[j][2] = load_at(K, p.ld, t, len, k0 + c, p.dimp);
        kv[j][3] = load_at(K, p.ld, t + 1, len, k0 + c, p.dimp);
    }
    __builtin_amdgcn_sched_barrier(0);
#pragma unroll
    for (int j = 0; j < 2; ++j) {
        const int idx = tid + 256 * j, c = (idx & 7) * 8, t = (idx >> 3) * 2;
        kv[j][0] = zero_outside(kv[j][0], t, len, v0 + c, p.vdimp);
        kv[j][1] = zero_outside(kv[j][1], t + 1, len, v0 + c, p.vdimp);
        kv[j][2] = zero_outside(kv[j][2], t, len, k0 + c, p.dimp);
        kv[j][3] = zero_outside(kv[j][3], t + 1, len, k0 + c, p.dimp);
        const u32x4 va = kv[j][0], vb = kv[j][1], ka = kv[j][2], kb = kv[j][3];
        const float pa = pw[max(len - 1 - t, 0)], pb = pw[max(len - 2 - t, 0)];  // (tokens past the end are zero)
        uint32_t o[8];
        pair_columns(va, vb, o);
#pragma unroll
        for (int e = 0; e < 8; ++e) *reinterpret_cast<uint32_t *>(lv + tile_at(c + e, t)) = o[e];
#pragma unroll
        for (int e = 0; e < 8; ++e) {
            const uint32_t xa = (e & 1) ? ka[e >> 1] & 0xffff0000u : ka[e >> 1] << 16, xb = (e & 1) ? kb[e >> 1] & 0xffff0000u : kb[e >> 1] << 16;
            uint32_t hi, lo;
            split2(__builtin_bit_cast(float, xa) * pa, __builtin_bit_cast(float, xb) * pb, hi, lo);
            *reinterpret_cast<uint32_t *>(kh + tile_at(c + e, t)) = hi;
            *reinterpret_cast<uint32_t *>(kl + tile_at(c + e, t)) = lo;
        }
    }
    __syncthreads();
    f32x4 acc[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) acc[i] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int ks = 0; ks < kLinBlock / 32; ++ks) {
        const bf16x8 a = *reinterpret_cast<const bf16x8 *>(lv + tile_at(wave * 16 + r16, ks * 32 + g * 8));
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            acc[i] = mfma_bf16(a, *reinterpret_cast<const bf16x8 *>(kh + tile_at(i * 16 + r16, ks * 32 + g * 8)), acc[i]);
            acc[i] = mfma_bf16(a, *reinterpret_cast<const bf16x8 *>(kl + tile_at(i * 16 + r16, ks * 32 + g * 8)), acc[i]);
        }
    }
    float *dst = w.sums + ((size_t)h * w.nb + blk) * p.vdimp * p.dimp;
#pragma unroll
    for (int i = 0; i < 4; ++i)
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            const int v = v0 + wave * 16 + g * 4 + e, k = k0 + i * 16 + r16;
            if (v < p.vdimp && k < p.dimp) dst[(size_t)v * p.dimp + k] = acc[i][e];
        }
}

// the state ahead of every block (as bf16 pairs) and after the last one (f32, in place)
__global__ __launch_bounds__(256) void k_linear_scan(LinearAttn p, LinearWs w) {
    const int h = blockIdx.y, e = blockIdx.x * 256 + threadIdx.x, size = p.vdimp * p.dimp;
    if (e >= size) return;
    const float *pw = p.decay_pow + (size_t)h * (kLinBlock + 1);
    float s = p.state[(size_t)h * size + e];
    const size_t base = (size_t)h * w.nb * size + e;
    constexpr int AH = 8;
    for (int b0 = 0; b0 < w.nb; b0 += AH) {
        float u[AH];
#pragma unroll
        for (int i = 0; i < AH; ++i) u[i] = b0 + i < w.nb ? w.sums[base + (size_t)(b0 + i) * size] : 0.f;
#pragma unroll
        for (int i = 0; i < AH; ++i) {
            if (b0 + i >= w.nb) break;
            const uint32_t b = __builtin_bit_cast(uint32_t, s);
            const float lo = s - __builtin_bit_cast(float, b & 0xffff0000u);
            w.hi[base + (size_t)(b0 + i) * size] = (uint16_t)(b >> 16);
            w.lo[base + (size_t)(b0 + i) * size] = (uint16_t)(__builtin_bit_cast(uint32_t, lo) >> 16);
            s = s * pw[min(kLinBlock, p.n - (b0 + i) * kLinBlock)] + u[i];
        }
    }
    p.state[(size_t)h * size + e] = s;
}

// o = d^(i + 1) S q_i + sum over j <= i of d^(i - j) (k_j . q_i) v_j; four waves of 32 queries
template <int NK, int NV>
__global__ __launch_bounds__(256, NV > 8 ? 1 : 2) void k_linear_out(LinearAttn p, LinearWs w) {
    extern __shared__ __attribute__((aligned(16))) uint8_t lds[];
    __shared__ float pw[2 * kLinBlock + 1];  // [kLinBlock + i] = decay^i, zero for i < 0
    constexpr int KS = NK * 64 + 16, QT = 2;
    uint8_t *lk = lds, *lv = lds + kLinBlock * KS;
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, r16 = lane & 15, g = lane >> 4;
    const int blk = blockIdx.x, h = blockIdx.y, t0 = blk * kLinBlock, len = min(kLinBlock, p.n - t0);
    const uint16_t *Q = (const uint16_t *)p.qkv + (size_t)h * p.dimp, *K = Q + (size_t)p.heads * p.dimp;
    const uint16_t *V = (const uint16_t *)p.qkv + 2 * (size_t)p.heads * p.dimp + (size_t)h * p.vdimp;
    Q += (size_t)t0 * p.ld, K += (size_t)t0 * p.ld, V += (size_t)t0 * p.ld;
    if (tid <= kLinBlock) pw[kLinBlock + tid] = p.decay_pow[(size_t)h * (kLinBlock + 1) + tid];
    if (tid < kLinBlock) pw[tid] = 0.f;
    bf16x8 q[QT][NK];
    int qi[QT];  // this lane's queries within the block
#pragma unroll
    for (int t = 0; t < QT; ++t) {
        qi[t] = wave * 32 + t * 16 + r16;
#pragma unroll
        for (int kk = 0; kk < NK; ++kk) q[t][kk] = __builtin_bit_cast(bf16x8, load_at(Q, p.ld, qi[t], len, kk * 32 + g * 8, p.dimp));
    }
#pragma unroll
    for (int half = 0; half < 2; ++half) {
        u32x4 kr[NK], vr[NV / 4][2];
        const int tk = half * 64 + (tid >> 2), tv = half * 64 + (tid >> 3) * 2;
#pragma unroll
        for (int j = 0; j < NK; ++j) kr[j] = load_at(K, p.ld, tk, len, j * 32 + (tid & 3) * 8, p.dimp);  // four threads per token
#pragma unroll
        for (int j = 0; j < NV / 4; ++j)  // eight threads per pair of tokens
#pragma unroll
            for (int e = 0; e < 2; ++e) vr[j][e] = load_at(V, p.ld, tv + e, len, j * 64 + (tid & 7) * 8, p.vdimp);
        __builtin_amdgcn_sched_barrier(0);
#pragma unroll
        for (int j = 0; j < NK; ++j) kr[j] = zero_outside(kr[j], tk, len, j * 32 + (tid & 3) * 8, p.dimp);
#pragma unroll
        for (int j = 0; j < NV / 4; ++j)
#pragma unroll
            for (int e = 0; e < 2; ++e) vr[j][e] = zero_outside(vr[j][e], tv + e, len, j * 64 + (tid & 7) * 8, p.vdimp);
#pragma unroll
        for (int j = 0; j < NK; ++j) *reinterpret_cast<u32x4 *>(lk + tk * KS + j * 64 + (tid & 3) * 16) = kr[j];
#pragma unroll
        for (int j = 0; j < NV / 4; ++j) {
            uint32_t o[8];
            pair_columns(vr[j][0], vr[j][1], o);
#pragma unroll
            for (int e = 0; e < 8; ++e) *reinterpret_cast<uint32_t *>(lv + tile_at(j * 64 + (tid & 7) * 8 + e, tv)) = o[e];
        }
    }
    // The state part: a value tile's operands are requested one tile ahead (the scheduling barriers keep hipcc from moving the
    // requests down to their uses, where each would wait for memory on its own).
#pragma unroll
    for (int t = 0; t < QT; ++t)
#pragma unroll
        for (int kk = 0; kk < NK; ++kk)
            q[t][kk] = __builtin_bit_cast(bf16x8, zero_outside(__builtin_bit_cast(u32x4, q[t][kk]), qi[t], len, kk * 32 + g * 8, p.dimp));
    f32x4 o[NV][QT];
    const size_t sb = ((size_t)h * w.nb + blk) * p.vdimp * p.dimp;
    bf16x8 hi[2][NK], lo[2][NK];
    auto request = [&](int v) {
#pragma unroll
        for (int kk = 0; kk < NK; ++kk) {
            // (rows past vdimp are never stored, columns past dimp meet a zero query: clamped addresses, no branches around the loads)
            const size_t at = sb + (size_t)min(v * 16 + r16, p.vdimp - 1) * p.dimp + min(kk * 32 + g * 8, p.dimp - 8);
            hi[v & 1][kk] = *reinterpret_cast<const bf16x8 *>(w.hi + at);
            lo[v & 1][kk] = *reinterpret_cast<const bf16x8 *>(w.lo + at);
        }
    };
    request(0);
#pragma unroll
    for (int v = 0; v < NV; ++v) {
        if (v + 1 < NV) request(v + 1);
        __builtin_amdgcn_sched_barrier(0);
#pragma unroll
        for (int t = 0; t < QT; ++t) o[v][t] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int kk = 0; kk < NK; ++kk)
#pragma unroll
            for (int t = 0; t < QT; ++t) {
                o[v][t] = mfma_bf16(hi[v & 1][kk], q[t][kk], o[v][t]);
                o[v][t] = mfma_bf16(lo[v & 1][kk], q[t][kk], o[v][t]);
            }
        __builtin_amdgcn_sched_barrier(0);
    }
    __syncthreads();
#pragma unroll
    for (int t = 0; t < QT; ++t) {
        const float di = pw[kLinBlock + qi[t] + 1];
#pragma unroll
        for (int v = 0; v < NV; ++v) o[v][t] *= di;
    }
    for (int kt = 0; kt <= 2 * wave + 1 && kt * 16 < len; kt += 2) {
        f32x4 s[2][QT];
#pragma unroll
        for (int j = 0; j < 2; ++j) {
#pragma unroll
            for (int t = 0; t < QT; ++t) s[j][t] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int kk = 0; kk < NK; ++kk) {
                const bf16x8 a = *reinterpret_cast<const bf16x8 *>(lk + ((kt + j) * 16 + r16) * KS + kk * 64 + g * 16);
#pragma unroll
                for (int t = 0; t < QT; ++t) s[j][t] = mfma_bf16(a, q[t][kk], s[j][t]);
            }
        }
        bf16x8 ph[QT], pl[QT];
#pragma unroll
        for (int t = 0; t < QT; ++t) {
            u32x4 hi, lo;
#pragma unroll
            for (int j = 0; j < 2; ++j)
#pragma unroll
                for (int e = 0; e < 4; ++e) s[j][t][e] *= pw[kLinBlock + qi[t] - ((kt + j) * 16 + g * 4 + e)];
#pragma unroll
            for (int j = 0; j < 4; ++j) {
                uint32_t uh, ul;
                split2(s[j >> 1][t][(j & 1) * 2], s[j >> 1][t][(j & 1) * 2 + 1], uh, ul);
                hi[j] = uh;
                lo[j] = ul;
            }
            ph[t] = __builtin_bit_cast(bf16x8, hi);
            pl[t] = __builtin_bit_cast(bf16x8, lo);
        }
#pragma unroll
        for (int v = 0; v < NV; ++v) {
            const u32x2 a0 = *reinterpret_cast<const u32x2 *>(lv + tile_at(v * 16 + r16, kt * 16 + g * 4));
            const u32x2 a1 = *reinterpret_cast<const u32x2 *>(lv + tile_at(v * 16 + r16, kt * 16 + 16 + g * 4));
            const bf16x8 a = __builtin_bit_cast(bf16x8, u32x4{a0.x, a0.y, a1.x, a1.y});
#pragma unroll
            for (int t = 0; t < QT; ++t) {
                o[v][t] = mfma_bf16(a, ph[t], o[v][t]);
                o[v][t] = mfma_bf16(a, pl[t], o[v][t]);
            }
        }
    }
#pragma unroll
    for (int t = 0; t < QT; ++t) {
        if (qi[t] >= len) continue;
        float *dst = p.out + (size_t)(t0 + qi[t]) * p.ldo + (size_t)h * p.vdimp + g * 4;
#pragma unroll
        for (int v = 0; v < NV; ++v)
            if (v * 16 < p.vdimp) *reinterpret_cast<f32x4 *>(dst + v * 16) = o[v][t];
    }
}

static int n_blocks(int n) { return (n + kLinBlock - 1) / kLinBlock; }
size_t linear_workspace_bytes(int n, int heads, int dimp, int vdimp) { return (size_t)n_blocks(n) * heads * dimp * vdimp * 8; }
bool linear_chunked_supported(int dimp, int vdimp) { return dimp % 32 == 0 && vdimp % 32 == 0 && dimp <= 256 && vdimp <= 256; }

template <int NK, int NV>
static hipError_t out_go(const LinearAttn &a, const LinearWs &w, hipStream_t s) {
    const size_t lds = (size_t)kLinBlock * (NK * 64 + 16) + (size_t)NV * 16 * kTileBytes;
    if (lds > 65536) {
        const hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void *>(k_linear_out<NK, NV>), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
        if (e != hipSuccess) return e;
    }
    hipLaunchKernelGGL((k_linear_out<NK, NV>), dim3(w.nb, a.heads), dim3(256), lds, s, a, w);
    return hipGetLastError();
}

hipError_t launch_linear_chunked(const LinearAttn &a, hipStream_t s) {
    if (!linear_chunked_supported(a.dimp, a.vdimp) || a.workspace_bytes < linear_workspace_bytes(a.n, a.heads, a.dimp, a.vdimp)) return hipErrorInvalidValue;
    LinearWs w;
    w.nb = n_blocks(a.n);
    const size_t cells = (size_t)w.nb * a.heads * a.dimp * a.vdimp;
    w.sums = (float *)a.workspace;
    w.hi = (uint16_t *)(w.sums + cells);
    w.lo = w.hi + cells;
    const int pieces = ((a.dimp + 63) / 64) * ((a.vdimp + 63) / 64);
    hipLaunchKernelGGL(k_linear_sums, dim3(w.nb, a.heads, pieces), dim3(256), 3 * 64 * kTileBytes, s, a, w);
    hipLaunchKernelGGL(k_linear_scan, dim3((a.dimp * a.vdimp + 255) / 256, a.heads), dim3(256), 0, s, a, w);
    const int nk = a.dimp / 32, nv = a.vdimp / 16;
    if (nk <= 2) return nv <= 4 ? out_go<2, 4>(a, w, s) : nv <= 8 ? out_go<2, 8>(a, w, s) : out_go<2, 16>(a, w, s);
    if (nk <= 4) return nv <= 4 ? out_go<4, 4>(a, w, s) : nv <= 8 ? out_go<4, 8>(a, w, s) : out_go<4, 16>(a, w, s);
    return nv <= 8 ? out_go<8, 8>(a, w, s) : out_go<8, 16>(a, w, s);
}

}  // namespace bitnet_hip
