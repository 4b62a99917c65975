// kernels_dense.hip -- operators on bf16 weight matrices (gfx950): embedding rows, residual + norm rows, the many-row matmul
// and the matrix-vector product of the decode step with its input transform folded in.
//
// Precision: residual stream, norms and accumulation are f32 everywhere.  The matmul multiplies bf16 activations on the matrix
// cores, or -- a_f32 -- f32 activations with f32 multiply-adds; the matrix-vector product always multiplies f32 activations.
#include <algorithm>

#include "dense.hpp"

namespace bitnet_hip {

// ---- embedding rows ---------------------------------------------------------------------------------------------------
__global__ void k_embed_bf16(const uint16_t *__restrict__ table, size_t ld, const int *__restrict__ tokens, const int *__restrict__ offset,
                             int width, int vocab, float scale, const float *__restrict__ norm_w, float eps, TokenPairs pairs, float *__restrict__ out) {
    __shared__ float slot[4];
    const int at = (offset ? *offset : 0) + blockIdx.x;
    auto token = [&](int i) { return min(max(tokens[i], 0), vocab - 1); };
    const int tok = token(at);
    if (pairs.table) {
        const uint64_t sum = (uint64_t)token(max(at - 1, 0)) * pairs.mul_prev + (uint64_t)tok * pairs.mul_cur;
        const uint64_t pair = at == 0 ? pairs.buckets : (sum | pairs.buckets) >> 32 ? sum % pairs.buckets : (uint32_t)sum % (uint32_t)pairs.buckets;
        const uint16_t *a = table + (size_t)tok * ld, *b = pairs.table + (size_t)pair * pairs.ld;
        float *o = out + (size_t)blockIdx.x * width;
        if (width % 4 == 0) {
            for (int i = 4 * (threadIdx.x + 256 * blockIdx.y); i < width; i += 1024 * gridDim.y) {
                const u32x2 x = *reinterpret_cast<const u32x2 *>(a + i), y = *reinterpret_cast<const u32x2 *>(b + i);
                *reinterpret_cast<f32x4 *>(o + i) = scale * f32x4{bf2f(x.x & 0xffffu), bf2f(x.x >> 16), bf2f(x.y & 0xffffu), bf2f(x.y >> 16)} +
                                                    f32x4{bf2f(y.x & 0xffffu), bf2f(y.x >> 16), bf2f(y.y & 0xffffu), bf2f(y.y >> 16)};
            }
        } else {
            for (int i = threadIdx.x + 256 * blockIdx.y; i < width; i += 256 * gridDim.y) o[i] = scale * bf2f(a[i]) + bf2f(b[i]);
        }
        return;
    }
    if (norm_w) {
        const uint16_t *row = table + (size_t)tok * ld;
        constexpr int NR = 16;  // rows of up to 4096 columns in registers, what lies behind is read again
        float ss = 0.f, v[NR], w[NR];
#pragma unroll
        for (int j = 0; j < NR; ++j) {
            const int i = threadIdx.x + 256 * j;
            v[j] = i < width ? scale * bf2f(row[i]) : 0.f;
            w[j] = i < width ? norm_w[i] : 0.f;
        }
#pragma unroll
        for (int j = 0; j < NR; ++j) ss += v[j] * v[j];
        for (int i = threadIdx.x + 256 * NR; i < width; i += 256) ss += scale * bf2f(row[i]) * (scale * bf2f(row[i]));
        const float inv = 1.0f / sqrtf(group_sum<4>(ss, slot) / (float)width + eps);
        float *o = out + (size_t)blockIdx.x * width;
#pragma unroll
        for (int j = 0; j < NR; ++j)
            if ((int)threadIdx.x + 256 * j < width) o[threadIdx.x + 256 * j] = v[j] * inv * w[j];
        for (int i = threadIdx.x + 256 * NR; i < width; i += 256) o[i] = scale * bf2f(row[i]) * inv * norm_w[i];
        return;
    }
    for (int i = threadIdx.x; i < width; i += blockDim.x) out[(size_t)blockIdx.x * width + i] = scale * bf2f(table[(size_t)tok * ld + i]);
}

hipError_t launch_embed_bf16(const uint16_t *table, size_t ld, const int *tokens, const int *offset, int n, int width, int vocab, float scale,
                             const float *norm_w, float eps, const TokenPairs &pairs, float *out, hipStream_t s) {
    const int parts = pairs.table && n == 1 ? (width + 1023) / 1024 : 1;  // (one token: its row at once)
    hipLaunchKernelGGL(k_embed_bf16, dim3(n, parts), dim3(256), 0, s, table, ld, tokens, offset, width, vocab, scale, norm_w, eps, pairs, out);
    return hipGetLastError();
}

__global__ void k_gather_rows(const float *__restrict__ x, const int *__restrict__ rows, int width, float *__restrict__ out) {
    const float *src = x + (size_t)rows[blockIdx.x] * width;
    for (int i = threadIdx.x; i < width; i += blockDim.x) out[(size_t)blockIdx.x * width + i] = src[i];
}

hipError_t launch_gather_rows(const float *x, const int *rows, int n, int width, float *out, hipStream_t s) {
    hipLaunchKernelGGL(k_gather_rows, dim3(n), dim3(256), 0, s, x, rows, width, out);
    return hipGetLastError();
}

// the last inputs of a portion into the ring of a causal convolution (position p in row p % taps)
template <class T>
__global__ __launch_bounds__(256) void k_conv_keep(const T *rows, size_t ld, int channels, int taps, float *ring, const int *pos_ptr, int n) {
    const int i = blockIdx.x * 256 + threadIdx.x, pos0 = *pos_ptr;
    if (i >= channels) return;
    for (int t = max(0, n - (taps - 1)); t < n; ++t) ring[(size_t)((pos0 + t) % taps) * channels + i] = ld_act(rows + (size_t)t * ld, i);
}

hipError_t launch_conv_keep(const void *rows, size_t ld, int rows_f32, int channels, int taps, float *ring, const int *pos, int n, hipStream_t s) {
    const dim3 grid((channels + 255) / 256);
    if (rows_f32)
        hipLaunchKernelGGL(k_conv_keep<float>, grid, dim3(256), 0, s, (const float *)rows, ld, channels, taps, ring, pos, n);
    else
        hipLaunchKernelGGL(k_conv_keep<uint16_t>, grid, dim3(256), 0, s, (const uint16_t *)rows, ld, channels, taps, ring, pos, n);
    return hipGetLastError();
}

// ---- residual + norm rows ---------------------------------------------------------------------------------------------
// x += scale * norm(y; post_w); h = norm(x; next_w), or x itself without next_w.  One workgroup per row; rows of up to 4096 columns stay in registers.
constexpr int kRowRegs = 16;

template <class TH>
__global__ __launch_bounds__(256) void k_residual_norm_rows(float *__restrict__ x, const float *__restrict__ y, size_t ldy, const float *__restrict__ post_w,
                                                            const float *__restrict__ scale, const float *__restrict__ next_w, float offset, float eps,
                                                            int width, TH *__restrict__ h, size_t ldh) {
    __shared__ float slot[4];
    const int tid = threadIdx.x;
    float *xr = x + (size_t)blockIdx.x * width;
    const float *yr = y ? y + (size_t)blockIdx.x * ldy : nullptr;
    const bool regs = width <= 256 * kRowRegs;
    float xv[kRowRegs];
    if (yr) {
        float ss = 0.f, yv[kRowRegs];
        if (regs) {
#pragma unroll
            for (int j = 0; j < kRowRegs; ++j) {
                const int i = tid + 256 * j;
                yv[j] = i < width ? yr[i] : 0.f;
                xv[j] = i < width ? xr[i] : 0.f;
                ss += yv[j] * yv[j];
            }
        } else {
            for (int i = tid; i < width; i += 256) ss += yr[i] * yr[i];
        }
        const float inv = 1.0f / sqrtf(group_sum<4>(ss, slot) / (float)width + eps);
        if (regs) {
#pragma unroll
            for (int j = 0; j < kRowRegs; ++j) {
                const int i = tid + 256 * j;
                if (i < width) {
                    xv[j] += (scale ? scale[i] : 1.0f) * (yv[j] * inv * (offset + post_w[i]));
                    xr[i] = xv[j];
                }
            }
        } else {
            for (int i = tid; i < width; i += 256) xr[i] += (scale ? scale[i] : 1.0f) * (yr[i] * inv * (offset + post_w[i]));
        }
    } else if (regs) {
#pragma unroll
        for (int j = 0; j < kRowRegs; ++j) xv[j] = tid + 256 * j < width ? xr[tid + 256 * j] : 0.f;
    }
    if (!h) return;
    float ss = 0.f;
    if (regs) {
#pragma unroll
        for (int j = 0; j < kRowRegs; ++j) ss += xv[j] * xv[j];
    } else {
        for (int i = tid; i < width; i += 256) ss += xr[i] * xr[i];
    }
    TH *hr = h + (size_t)blockIdx.x * ldh;
    if (!next_w) {
        if (regs) {
#pragma unroll
            for (int j = 0; j < kRowRegs; ++j)
                if (tid + 256 * j < width) st_act(hr, tid + 256 * j, xv[j]);
        } else {
            for (int i = tid; i < width; i += 256) st_act(hr, i, xr[i]);
        }
        for (int i = width + tid; i < (int)ldh; i += 256) st_act(hr, i, 0.f);
        return;
    }
    const float inv = 1.0f / sqrtf(group_sum<4>(ss, slot) / (float)width + eps);
    if (regs) {
#pragma unroll
        for (int j = 0; j < kRowRegs; ++j) {
            const int i = tid + 256 * j;
            if (i < width) st_act(hr, i, xv[j] * inv * (offset + next_w[i]));
        }
    } else {
        for (int i = tid; i < width; i += 256) st_act(hr, i, xr[i] * inv * (offset + next_w[i]));
    }
    for (int i = width + tid; i < (int)ldh; i += 256) st_act(hr, i, 0.f);
}

hipError_t launch_residual_norm_rows(float *x, const float *y, size_t ldy, const float *post_w, const float *scale, const float *next_w,
                                     float offset, float eps, int m, int width, void *h, size_t ldh, int h_f32, hipStream_t s) {
    if (h_f32)
        hipLaunchKernelGGL(k_residual_norm_rows<float>, dim3(m), dim3(256), 0, s, x, y, ldy, post_w, scale, next_w, offset, eps, width, (float *)h, ldh);
    else
        hipLaunchKernelGGL(k_residual_norm_rows<uint16_t>, dim3(m), dim3(256), 0, s, x, y, ldy, post_w, scale, next_w, offset, eps, width, (uint16_t *)h, ldh);
    return hipGetLastError();
}

// Rows of a block whose sublayers add up: t = y + the chosen experts' rows, x += mult * t or scale * norm(t); h = norm(x), x or [x; x2].  Four columns at a time, rows of up to
// 4096 columns in registers.
__device__ __forceinline__ f32x4 ld4(const float *p, size_t i) { return *reinterpret_cast<const f32x4 *>(p + i); }
__device__ __forceinline__ f32x4 ld4(const uint16_t *p, size_t i) {
    const u32x2 v = *reinterpret_cast<const u32x2 *>(p + i);
    return f32x4{bf2f(v.x & 0xffffu), bf2f(v.x >> 16), bf2f(v.y & 0xffffu), bf2f(v.y >> 16)};
}
__device__ __forceinline__ void st4(float *p, size_t i, f32x4 v) { *reinterpret_cast<f32x4 *>(p + i) = v; }
__device__ __forceinline__ void st4(uint16_t *p, size_t i, f32x4 v) {
    *reinterpret_cast<bf16x4 *>(p + i) = bf16x4{(__bf16)v.x, (__bf16)v.y, (__bf16)v.z, (__bf16)v.w};
}
constexpr int kSumRegs = 4;

// IDENTITY: slots may be negative.  GATED: with a number per row on y, a gate per column on what is added, or both.
template <class T, bool VEC, bool IDENTITY, bool GATED>
__global__ __launch_bounds__(256) void k_sum_norm_rows(SumRows p) {
    __shared__ float slot[4];
    const int tid = threadIdx.x, width = (int)p.width;
    float *x = p.x + (size_t)blockIdx.x * width;
    const float *y = p.y ? p.y + (size_t)blockIdx.x * p.ldy : nullptr;
    T *h = p.h ? (T *)p.h + (size_t)blockIdx.x * p.ldh : nullptr;
    const T *er = (const T *)p.expert_rows;
    const int *slots = p.slots + (size_t)blockIdx.x * p.top;
    const float *sw = p.slot_weights + (size_t)blockIdx.x * p.top;
    const float *x2 = p.x2 ? p.x2 + (size_t)blockIdx.x * width : nullptr;
    const T *gate = GATED && p.gate ? (const T *)p.gate + (size_t)blockIdx.x * p.ld_gate : nullptr;
    const float ys = GATED && p.y_scale ? p.y_scale[(size_t)blockIdx.x * p.ld_y_scale] : 1.0f;
    const T *input = p.input ? (const T *)p.input + (size_t)blockIdx.x * p.ld_input : nullptr;  // (may be h: a thread reads its columns ahead of writing them)
    const int top = (int)p.top;
    if (VEC) {
        f32x4 v[kSumRegs];
        const int n4 = width >> 2;
#pragma unroll
        for (int j = 0; j < kSumRegs; ++j) {
            const int i = tid + 256 * j;
            v[j] = f32x4{0.f, 0.f, 0.f, 0.f};
            if (i < n4) v[j] = ld4(x, 4 * i);
        }
        if (y || top) {
            f32x4 a[kSumRegs];
#pragma unroll
            for (int j = 0; j < kSumRegs; ++j) {
                const int i = tid + 256 * j;
                a[j] = f32x4{0.f, 0.f, 0.f, 0.f};
                if (y && i < n4) a[j] = ld4(y, 4 * i);
                if (GATED) a[j] *= ys;
            }
            float through = 0.f;
#pragma unroll 4
            for (int k = 0; k < top; ++k) {
                const float w = sw[k];
                const T *row;
                if (IDENTITY) {  // (without a branch: an identity's place is taken by some row, which is not added)
                    const int s = slots[k];
                    row = er + (size_t)max(s, 0) * p.ld_expert;
                    through += s < 0 ? w : 0.f;
#pragma unroll
                    for (int j = 0; j < kSumRegs; ++j) {
                        const int i = tid + 256 * j;
                        const f32x4 e = ld4(row, 4 * min(i, n4 - 1));
                        a[j] += s < 0 || i >= n4 ? f32x4{0.f, 0.f, 0.f, 0.f} : w * e;
                    }
                    continue;
                }
                row = er + (size_t)slots[k] * p.ld_expert;
#pragma unroll
                for (int j = 0; j < kSumRegs; ++j) {
                    const int i = tid + 256 * j;
                    const f32x4 e = ld4(row, 4 * min(i, n4 - 1));  // (no branch around the load: the rows' loads overlap)
                    a[j] += i < n4 ? w * e : f32x4{0.f, 0.f, 0.f, 0.f};
                }
            }
            if (IDENTITY && through != 0.f) {
#pragma unroll
                for (int j = 0; j < kSumRegs; ++j) {
                    const int i = tid + 256 * j;
                    if (i < n4) a[j] += through * (input ? ld4(input, 4 * i) : v[j]);
                }
            }
            float post = 0.f;
            if (p.post_weight) {
                float ss = 0.f;
#pragma unroll
                for (int j = 0; j < kSumRegs; ++j) ss += (a[j].x * a[j].x + a[j].y * a[j].y) + (a[j].z * a[j].z + a[j].w * a[j].w);
                post = 1.0f / sqrtf(group_sum<4>(ss, slot) / (float)width + p.eps);
            }
#pragma unroll
            for (int j = 0; j < kSumRegs; ++j) {
                const int i = tid + 256 * j;
                if (i < n4) {
                    if (GATED && gate) a[j] *= ld4(gate, 4 * i);
                    if (p.post_weight) {
                        f32x4 r = a[j] * post * (p.weight_offset + ld4(p.post_weight, 4 * i));
                        if (p.scale) r *= ld4(p.scale, 4 * i);
                        v[j] += r;
                    } else {
                        v[j] += p.mult * a[j];
                    }
                    st4(x, 4 * i, v[j]);
                }
            }
        }
        if (!h) return;
        if (x2) {
#pragma unroll
            for (int j = 0; j < kSumRegs; ++j) {
                const int i = tid + 256 * j;
                if (i < n4) {
                    st4(h, 4 * i, v[j]);
                    st4(h, width + 4 * i, ld4(x2, 4 * i));
                }
            }
        } else if (!p.weight) {
#pragma unroll
            for (int j = 0; j < kSumRegs; ++j)
                if (tid + 256 * j < n4) st4(h, 4 * (tid + 256 * j), v[j]);
        } else {
            float mean = 0.f, ss = 0.f;
            if (p.center) {
                float t = 0.f;
#pragma unroll
                for (int j = 0; j < kSumRegs; ++j) t += (v[j].x + v[j].y) + (v[j].z + v[j].w);
                mean = group_sum<4>(t, slot) / (float)width;
            }
#pragma unroll
            for (int j = 0; j < kSumRegs; ++j) {
                if (tid + 256 * j < n4) v[j] -= mean;
                ss += (v[j].x * v[j].x + v[j].y * v[j].y) + (v[j].z * v[j].z + v[j].w * v[j].w);
            }
            const float inv = 1.0f / sqrtf(group_sum<4>(ss, slot) / (float)width + p.eps);
#pragma unroll
            for (int j = 0; j < kSumRegs; ++j) {
                const int i = tid + 256 * j;
                if (i < n4) {
                    f32x4 r = v[j] * inv * (p.weight_offset + ld4(p.weight, 4 * i));
                    if (p.bias) r += ld4(p.bias, 4 * i);
                    st4(h, 4 * i, r);
                }
            }
        }
    } else {  // (a thread comes back to its own columns only)
        if (y || top) {
            auto sum = [&](int i) {
                float a = y ? ys * y[i] : 0.f;
                for (int k = 0; k < top; ++k) a += sw[k] * (!IDENTITY || slots[k] >= 0 ? ld_act(er + (size_t)slots[k] * p.ld_expert, i) : input ? ld_act(input, i) : x[i]);
                return a;
            };
            float post = 0.f;
            if (p.post_weight) {
                float ss = 0.f;
                for (int i = tid; i < width; i += 256) {
                    const float a = sum(i);
                    ss += a * a;
                }
                post = 1.0f / sqrtf(group_sum<4>(ss, slot) / (float)width + p.eps);
            }
            for (int i = tid; i < width; i += 256)
                x[i] += (gate ? ld_act(gate, i) : 1.0f) *
                        (p.post_weight ? (p.scale ? p.scale[i] : 1.0f) * (sum(i) * post * (p.weight_offset + p.post_weight[i])) : p.mult * sum(i));
        }
        if (!h) return;
        if (x2) {
            for (int i = tid; i < width; i += 256) {
                st_act(h, i, x[i]);
                st_act(h, width + i, x2[i]);
            }
        } else if (!p.weight) {
            for (int i = tid; i < width; i += 256) st_act(h, i, x[i]);
        } else {
            float mean = 0.f, ss = 0.f;
            if (p.center) {
                float t = 0.f;
                for (int i = tid; i < width; i += 256) t += x[i];
                mean = group_sum<4>(t, slot) / (float)width;
            }
            for (int i = tid; i < width; i += 256) ss += (x[i] - mean) * (x[i] - mean);
            const float inv = 1.0f / sqrtf(group_sum<4>(ss, slot) / (float)width + p.eps);
            for (int i = tid; i < width; i += 256) st_act(h, i, (x[i] - mean) * inv * (p.weight_offset + p.weight[i]) + (p.bias ? p.bias[i] : 0.f));
        }
    }
    for (int i = (x2 ? 2 : 1) * width + tid; i < (int)p.ldh; i += 256) st_act(h, i, 0.f);
}

hipError_t launch_sum_norm_rows(const SumRows &a, hipStream_t s) {
    // (four columns at a time: every row of every operand starts on its own alignment)
    const bool vec = a.width % 4 == 0 && a.width <= 1024 * kSumRegs && a.ldy % 4 == 0 && a.ld_expert % 4 == 0 && a.ldh % 4 == 0 && a.ld_input % 4 == 0 && a.ld_gate % 4 == 0;
    auto go = [&](auto plain, auto identity, auto gated, auto both) {
        const bool g = a.gate || a.y_scale;
        hipLaunchKernelGGL(a.identity ? (g ? both : identity) : g ? gated : plain, dim3(a.m), dim3(256), 0, s, a);
        return hipGetLastError();
    };
    if (a.h_f32)
        return vec ? go(k_sum_norm_rows<float, true, false, false>, k_sum_norm_rows<float, true, true, false>, k_sum_norm_rows<float, true, false, true>, k_sum_norm_rows<float, true, true, true>)
                   : go(k_sum_norm_rows<float, false, false, false>, k_sum_norm_rows<float, false, true, false>, k_sum_norm_rows<float, false, false, true>,
                        k_sum_norm_rows<float, false, true, true>);
    return vec ? go(k_sum_norm_rows<uint16_t, true, false, false>, k_sum_norm_rows<uint16_t, true, true, false>, k_sum_norm_rows<uint16_t, true, false, true>,
                    k_sum_norm_rows<uint16_t, true, true, true>)
               : go(k_sum_norm_rows<uint16_t, false, false, false>, k_sum_norm_rows<uint16_t, false, true, false>, k_sum_norm_rows<uint16_t, false, false, true>,
                    k_sum_norm_rows<uint16_t, false, true, true>);
}

// h = norm(o; w) * gate (gate: already through its sigmoid); the mean runs over mean_n elements, padding columns of o are zero
template <class TG, class TH>
__global__ __launch_bounds__(256) void k_gated_norm_rows(const float *__restrict__ o, size_t ldo, const float *__restrict__ w, const TG *__restrict__ gate,
                                                         size_t ldg, float eps, int n, int mean_n, TH *__restrict__ h, size_t ldh) {
    __shared__ float slot[4];
    const int tid = threadIdx.x;
    const float *orow = o + (size_t)blockIdx.x * ldo;
    const TG *grow = gate + (size_t)blockIdx.x * ldg;
    TH *hr = h + (size_t)blockIdx.x * ldh;
    float ss = 0.f;
    for (int i = tid; i < n; i += 256) ss += orow[i] * orow[i];
    const float inv = 1.0f / sqrtf(group_sum<4>(ss, slot) / (float)mean_n + eps);
    for (int i = tid; i < n; i += 256) st_act(hr, i, orow[i] * inv * w[i] * ld_act(grow, i));
    for (int i = n + tid; i < (int)ldh; i += 256) st_act(hr, i, 0.f);
}

hipError_t launch_gated_norm_rows(const float *o, size_t ldo, const float *w, const void *gate, size_t ldg, int gate_f32, float eps, int m, int n,
                                  int mean_n, void *h, size_t ldh, int h_f32, hipStream_t s) {
    auto go = [&](auto *fn, auto *g, auto *out) { hipLaunchKernelGGL(fn, dim3(m), dim3(256), 0, s, o, ldo, w, g, ldg, eps, n, mean_n, out, ldh); };
    if (gate_f32 && h_f32)
        go(k_gated_norm_rows<float, float>, (const float *)gate, (float *)h);
    else if (gate_f32)
        go(k_gated_norm_rows<float, uint16_t>, (const float *)gate, (uint16_t *)h);
    else if (!h_f32)
        go(k_gated_norm_rows<uint16_t, uint16_t>, (const uint16_t *)gate, (uint16_t *)h);
    else
        return hipErrorInvalidValue;
    return hipGetLastError();
}

// ---- latent rows ------------------------------------------------------------------------------------------------------
template <class T>
__device__ void latent_row(const LatentRows &p, int row, float *slot) {
    const int tid = threadIdx.x;
    const float *z = p.z + (size_t)row * p.ldz;
    if (p.cq) {
        float ss = 0.f;
        for (int i = tid; i < p.q_rank; i += 256) ss += z[i] * z[i];
        const float inv = 1.0f / sqrtf(group_sum<4>(ss, slot) / (float)p.q_rank + p.eps);
        T *o = (T *)p.cq + (size_t)row * p.ldcq;
        for (int i = tid; i < p.ldcq; i += 256) st_act(o, i, i < p.q_rank ? z[i] * inv * p.q_weight[i] : 0.f);
    }
    if (p.kv_rank == 0) return;
    const int pos = *p.pos + row;
    const float *zc = z + p.q_rank, *zr = zc + p.kv_rank;
    float ss = 0.f;
    for (int i = tid; i < p.kv_rank; i += 256) ss += zc[i] * zc[i];
    const float inv = 1.0f / sqrtf(group_sum<4>(ss, slot) / (float)p.kv_rank + p.eps);
    T *c = (T *)p.ccache + (size_t)pos * p.ldc;
    for (int i = tid; i < p.kv_rank; i += 256) st_act(c, i, zc[i] * inv * p.kv_weight[i]);
    const int half = p.rot_dim / 2;
    T *r = (T *)p.rcache + (size_t)pos * p.ldr;
    for (int i = tid; i < half; i += 256) {
        const float cs = p.rope_cos[(size_t)pos * half + i], sn = p.rope_sin[(size_t)pos * half + i];
        const float u = zr[i], v = zr[i + half];
        st_act(r, i, u * cs - v * sn);
        st_act(r, i + half, v * cs + u * sn);
    }
}

template <class T>
__global__ __launch_bounds__(256) void k_latent_rows(LatentRows p) {
    __shared__ float slot[4];
    latent_row<T>(p, blockIdx.x, slot);
}

hipError_t launch_latent_rows(const LatentRows &a, hipStream_t s) {
    if (a.f32)
        hipLaunchKernelGGL(k_latent_rows<float>, dim3(a.m), dim3(256), 0, s, a);
    else
        hipLaunchKernelGGL(k_latent_rows<uint16_t>, dim3(a.m), dim3(256), 0, s, a);
    return hipGetLastError();
}

// ---- matrix-vector product --------------------------------------------------------------------------------------------
// One launch per product of the decode step.  Every workgroup forms the whole input vector (L2-resident, a few KiB) in LDS --
// norm, residual + norm, or gated norm -- then its waves take rows: LPR lanes per row, 16 bytes of weights per lane and chunk,
// R rows x U chunks in flight.  The first block of weights is requested ahead of the input transform.
struct GemvK {
    GemvArgs a;
    LatentRows lat;
    int kp;        // columns rounded up to whole LPR * 8 * U steps: length of the LDS vector
    int groups;    // row groups (R * 64 / LPR rows each) of one batch member
    int lat_wg;    // workgroup index that writes the latent row, or -1
};

template <bool MORE>
__device__ void form_input(const VecIn &in, const float *x, int cols, int kp, float *xs, float *slot, bool writer) {
    const int tid = threadIdx.x;
    const int n = in.n;
    if (in.kind == BITNET_HIP_IN_PLAIN) {
        if ((cols & 3) == 0 && ((uintptr_t)x & 15) == 0) {
            constexpr int NV = 8;  // sixteen-byte loads in flight per thread
            const int c4 = cols >> 2, k4 = kp >> 2;
            for (int i0 = tid; i0 < k4; i0 += 256 * NV) {
                f32x4 v[NV];
#pragma unroll
                for (int j = 0; j < NV; ++j) v[j] = reinterpret_cast<const f32x4 *>(x)[min(i0 + 256 * j, c4 - 1)];
#pragma unroll
                for (int j = 0; j < NV; ++j) {
                    const int i = i0 + 256 * j;
                    if (i < k4) reinterpret_cast<f32x4 *>(xs)[i] = i < c4 ? v[j] : f32x4{0.f, 0.f, 0.f, 0.f};
                }
            }
        } else {
            for (int i = tid; i < kp; i += 256) xs[i] = i < cols ? x[i] : 0.f;
        }
        __syncthreads();
        return;
    }
    constexpr int NR = 4;  // float4 registers: vectors of up to 4096 elements
    if ((n & 3) == 0 && n <= 1024 * NR) {
        f32x4 xv[NR];
        const int n4 = n >> 2;
#pragma unroll
        for (int j = 0; j < NR; ++j) {
            const int i = tid + 256 * j;
            const f32x4 v = reinterpret_cast<const f32x4 *>(x)[min(i, n4 - 1)];
            xv[j] = v * (i < n4 ? 1.0f : 0.0f);
        }
        if (in.kind >= BITNET_HIP_IN_RESIDUAL_NORM && in.y && !in.post_weight) {
            f32x4 yv[NR], yg[NR];
#pragma unroll
            for (int j = 0; j < NR; ++j) {
                yv[j] = reinterpret_cast<const f32x4 *>(in.y)[min(tid + 256 * j, n4 - 1)];
                yg[j] = MORE && in.y_gate ? reinterpret_cast<const f32x4 *>(in.y_gate)[min(tid + 256 * j, n4 - 1)] : f32x4{1.f, 1.f, 1.f, 1.f};
            }
#pragma unroll
            for (int j = 0; j < NR; ++j) {
                const int i = tid + 256 * j;
                if (i >= n4) continue;
                xv[j] += in.mult * yv[j] * yg[j];
                if (writer && in.x_out) reinterpret_cast<f32x4 *>(in.x_out)[i] = xv[j];
            }
        } else if (in.kind >= BITNET_HIP_IN_RESIDUAL_NORM && in.y) {
            f32x4 yv[NR], pw[NR], sc[NR];
            float ss = 0.f;
#pragma unroll
            for (int j = 0; j < NR; ++j) {
                const int i = tid + 256 * j;
                const int c = min(i, n4 - 1);
                const f32x4 v = reinterpret_cast<const f32x4 *>(in.y)[c];
                yv[j] = v * (i < n4 ? 1.0f : 0.0f);
                pw[j] = reinterpret_cast<const f32x4 *>(in.post_weight)[c];
            }
            if (in.scale) {
#pragma unroll
                for (int j = 0; j < NR; ++j) sc[j] = reinterpret_cast<const f32x4 *>(in.scale)[min(tid + 256 * j, n4 - 1)];
            } else {
#pragma unroll
                for (int j = 0; j < NR; ++j) sc[j] = f32x4{1.f, 1.f, 1.f, 1.f};
            }
            if (MORE && in.y_gate)
#pragma unroll
                for (int j = 0; j < NR; ++j) sc[j] *= reinterpret_cast<const f32x4 *>(in.y_gate)[min(tid + 256 * j, n4 - 1)];
#pragma unroll
            for (int j = 0; j < NR; ++j) ss += yv[j].x * yv[j].x + yv[j].y * yv[j].y + yv[j].z * yv[j].z + yv[j].w * yv[j].w;
            const float inv = 1.0f / sqrtf(group_sum<4>(ss, slot) / (float)in.mean_n + in.eps);
#pragma unroll
            for (int j = 0; j < NR; ++j) {
                const int i = tid + 256 * j;
                if (i >= n4) continue;
                xv[j] += sc[j] * (yv[j] * inv * (in.offset + pw[j]));
                if (writer && in.x_out) reinterpret_cast<f32x4 *>(in.x_out)[i] = xv[j];
            }
        }
        if (in.kind >= BITNET_HIP_IN_CONCAT) {
            const bool two = in.kind == BITNET_HIP_IN_CONCAT;
#pragma unroll
            for (int j = 0; j < NR; ++j) {
                const int i = tid + 256 * j;
                if (i >= n4) continue;
                reinterpret_cast<f32x4 *>(xs)[i] = xv[j];
                if (two) reinterpret_cast<f32x4 *>(xs)[n4 + i] = reinterpret_cast<const f32x4 *>(in.x2)[i];
            }
            for (int i = (two ? 2 : 1) * n + tid; i < kp; i += 256) xs[i] = 0.f;
            __syncthreads();
            return;
        }
        f32x4 bv[NR];
        if (in.center) {
            float t = 0.f;
#pragma unroll
            for (int j = 0; j < NR; ++j) {
                t += (xv[j].x + xv[j].y) + (xv[j].z + xv[j].w);
                bv[j] = in.bias ? reinterpret_cast<const f32x4 *>(in.bias)[min(tid + 256 * j, n4 - 1)] : f32x4{0.f, 0.f, 0.f, 0.f};
            }
            const float mean = group_sum<4>(t, slot) / (float)in.mean_n;
#pragma unroll
            for (int j = 0; j < NR; ++j) xv[j] -= tid + 256 * j < n4 ? mean : 0.f;
        }
        f32x4 wv[NR], gv[NR];
        float ss = 0.f;
#pragma unroll
        for (int j = 0; j < NR; ++j) {
            const int i = tid + 256 * j;
            wv[j] = reinterpret_cast<const f32x4 *>(in.weight)[min(i, n4 - 1)];
            ss += xv[j].x * xv[j].x + xv[j].y * xv[j].y + xv[j].z * xv[j].z + xv[j].w * xv[j].w;
        }
        if (in.gate) {
#pragma unroll
            for (int j = 0; j < NR; ++j) gv[j] = reinterpret_cast<const f32x4 *>(in.gate)[min(tid + 256 * j, n4 - 1)];
        } else {
#pragma unroll
            for (int j = 0; j < NR; ++j) gv[j] = f32x4{1.f, 1.f, 1.f, 1.f};
        }
        const float inv = 1.0f / sqrtf(group_sum<4>(ss, slot) / (float)in.mean_n + in.eps);
#pragma unroll
        for (int j = 0; j < NR; ++j) {
            const int i = tid + 256 * j;
            if (i >= n4) continue;
            f32x4 r = xv[j] * inv * (in.offset + wv[j]) * gv[j];
            if (in.center) r += bv[j];
            reinterpret_cast<f32x4 *>(xs)[i] = r;
            if (writer && in.h_out) reinterpret_cast<f32x4 *>(in.h_out)[i] = r;
        }
    } else {
        float ss = 0.f;
        if (in.kind >= BITNET_HIP_IN_RESIDUAL_NORM && in.y && !in.post_weight) {
            for (int i = tid; i < n; i += 256) {
                const float v = x[i] + in.mult * in.y[i] * (MORE && in.y_gate ? in.y_gate[i] : 1.0f);
                xs[i] = v;
                if (writer && in.x_out) in.x_out[i] = v;
                ss += v * v;
            }
        } else if (in.kind >= BITNET_HIP_IN_RESIDUAL_NORM && in.y) {
            for (int i = tid; i < n; i += 256) ss += in.y[i] * in.y[i];
            const float inv = 1.0f / sqrtf(group_sum<4>(ss, slot) / (float)in.mean_n + in.eps);
            ss = 0.f;
            for (int i = tid; i < n; i += 256) {
                const float v = x[i] + (in.scale ? in.scale[i] : 1.0f) * (MORE && in.y_gate ? in.y_gate[i] : 1.0f) * (in.y[i] * inv * (in.offset + in.post_weight[i]));
                xs[i] = v;
                if (writer && in.x_out) in.x_out[i] = v;
                ss += v * v;
            }
        } else {
            for (int i = tid; i < n; i += 256) {
                xs[i] = x[i];
                ss += x[i] * x[i];
            }
        }
        if (in.kind >= BITNET_HIP_IN_CONCAT) {
            const bool two = in.kind == BITNET_HIP_IN_CONCAT;
            for (int i = tid; two && i < n; i += 256) xs[n + i] = in.x2[i];
            for (int i = (two ? 2 : 1) * n + tid; i < kp; i += 256) xs[i] = 0.f;
            __syncthreads();
            return;
        }
        if (in.center) {  // (a thread comes back to its own elements only)
            float t = 0.f;
            for (int i = tid; i < n; i += 256) t += xs[i];
            const float mean = group_sum<4>(t, slot) / (float)in.mean_n;
            ss = 0.f;
            for (int i = tid; i < n; i += 256) {
                xs[i] -= mean;
                ss += xs[i] * xs[i];
            }
        }
        const float inv = 1.0f / sqrtf(group_sum<4>(ss, slot) / (float)in.mean_n + in.eps);
        for (int i = tid; i < n; i += 256) {
            xs[i] = xs[i] * inv * (in.offset + in.weight[i]) * (in.gate ? in.gate[i] : 1.0f) + (in.center && in.bias ? in.bias[i] : 0.f);
            if (writer && in.h_out) in.h_out[i] = xs[i];
        }
    }
    for (int i = n + tid; i < kp; i += 256) xs[i] = 0.f;
    __syncthreads();
}

template <int LPR>
__device__ __forceinline__ float lanes_total(float v) {
    if (LPR == 8) {
        v += dpp<0x141>(v);       // row_half_mirror
        v += dpp<0xb1>(v);        // quad_perm [1,0,3,2]
        return v + dpp<0x4e>(v);  // quad_perm [2,3,0,1]
    }
    v = row_sum(v);
    return LPR == 64 ? rows_sum(v) : v;
}

// MORE: whatever bitnet_hip_epilogue and a gate on the residual ask for
template <int LPR, int R, int U, bool MORE>
__global__ __launch_bounds__(256) void k_dense_gemv(GemvK p) {
    extern __shared__ __attribute__((aligned(16))) float xs[];
    __shared__ float slot[4];
    __shared__ float wbv[4];
    __shared__ int wbi[4];
    const GemvArgs &a = p.a;
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    if ((int)blockIdx.x == p.lat_wg) {  // (the whole workgroup)
        if (blockIdx.y > 0) return;
        if (p.lat.f32)
            latent_row<float>(p.lat, 0, slot);
        else
            latent_row<uint16_t>(p.lat, 0, slot);
        return;
    }
    const int n_wg = p.lat_wg >= 0 ? p.lat_wg : (int)gridDim.x;
    const int b = blockIdx.y;
    const int sub = lane / LPR, l = lane % LPR;
    constexpr int G = 64 / LPR;
    const uint16_t *wb = a.w + (size_t)b * a.w_batch;
    const int step = LPR * 8 * U;
    const int last_col = a.cols - 8;
    int g = blockIdx.x * 4 + wave;
    u32x4 w[R][U];
    auto fetch = [&](int grp, int k0) {
        const int row0 = (grp * G + sub) * R;
#pragma unroll
        for (int r = 0; r < R; ++r) {
            const int row = row0 + r < a.rows ? row0 + r : a.rows - 1;
            const uint16_t *wr = wb + (size_t)row * a.ld;
#pragma unroll
            for (int u = 0; u < U; ++u) {
                const int col = k0 + (u * LPR + l) * 8;
                w[r][u] = __builtin_nontemporal_load(reinterpret_cast<const u32x4 *>(wr + (col < last_col ? col : last_col)));
            }
        }
    };
    // the earlier positions of a convolution's rows, a tap per lane; summed behind the product
    const Epilogue &e = a.more;
    const bool conv = MORE && e.conv, mul = MORE && e.mul;
    const int pos = conv ? *e.pos : 0, mul_at = mul ? *e.mul_at : 0;
    float past[R];
    auto fetch_past = [&](int grp) {
#pragma unroll
        for (int r = 0; r < R; ++r) {
            const int ch = (grp * G + sub) * R + r - e.conv_from;
            past[r] = 0.f;
            if (ch < 0 || ch >= e.channels) continue;
            for (int j = l; j < e.taps - 1; j += LPR) {
                const int at = pos - (e.taps - 1) + j;
                if (at >= 0) past[r] += e.conv[(size_t)j * e.channels + ch] * e.ring[(size_t)(at % e.taps) * e.channels + ch];
            }
        }
    };
    if (g < p.groups) fetch(g, 0);
    if (conv && g < p.groups) fetch_past(g);
    form_input<MORE>(a.in, a.in.x + (size_t)b * a.x_batch, a.cols, p.kp, xs, slot, blockIdx.x == 0 && b == 0);
    float bv = -INFINITY;
    int bi = 0x7fffffff;
    for (; g < p.groups; g += n_wg * 4) {
        float acc[R];
#pragma unroll
        for (int r = 0; r < R; ++r) acc[r] = 0.f;
        for (int k0 = 0; k0 < p.kp; k0 += step) {
            u32x4 c[R][U];
#pragma unroll
            for (int r = 0; r < R; ++r)
#pragma unroll
                for (int u = 0; u < U; ++u) c[r][u] = w[r][u];
            if (k0 + step < p.kp)
                fetch(g, k0 + step);
            else if (g + n_wg * 4 < p.groups)
                fetch(g + n_wg * 4, 0);
#pragma unroll
            for (int u = 0; u < U; ++u) {
                const f32x4 x0 = *reinterpret_cast<const f32x4 *>(xs + k0 + (u * LPR + l) * 8);
                const f32x4 x1 = *reinterpret_cast<const f32x4 *>(xs + k0 + (u * LPR + l) * 8 + 4);
#pragma unroll
                for (int r = 0; r < R; ++r) {
                    const u32x4 v = c[r][u];
                    acc[r] = fmaf(x0.x, __builtin_bit_cast(float, v.x << 16), acc[r]);
                    acc[r] = fmaf(x0.y, __builtin_bit_cast(float, v.x & 0xffff0000u), acc[r]);
                    acc[r] = fmaf(x0.z, __builtin_bit_cast(float, v.y << 16), acc[r]);
                    acc[r] = fmaf(x0.w, __builtin_bit_cast(float, v.y & 0xffff0000u), acc[r]);
                    acc[r] = fmaf(x1.x, __builtin_bit_cast(float, v.z << 16), acc[r]);
                    acc[r] = fmaf(x1.y, __builtin_bit_cast(float, v.z & 0xffff0000u), acc[r]);
                    acc[r] = fmaf(x1.z, __builtin_bit_cast(float, v.w << 16), acc[r]);
                    acc[r] = fmaf(x1.w, __builtin_bit_cast(float, v.w & 0xffff0000u), acc[r]);
                }
            }
        }
        const int row0 = (g * G + sub) * R;
#pragma unroll
        for (int r = 0; r < R; ++r) acc[r] = lanes_total<LPR>(acc[r]);
        if (conv) {
            float f[R];
#pragma unroll
            for (int r = 0; r < R; ++r) f[r] = lanes_total<LPR>(past[r]);
#pragma unroll
            for (int r = 0; r < R; ++r) {
                const int row = row0 + r, ch = row - e.conv_from;
                if (ch < 0 || ch >= e.channels || row >= a.rows) continue;
                if (a.bias) acc[r] += a.bias[row];
                if (l == 0) e.ring[(size_t)(pos % e.taps) * e.channels + ch] = acc[r];  // (no earlier position's slot)
                acc[r] = acc[r] * e.conv[(size_t)(e.taps - 1) * e.channels + ch] + f[r];
            }
            if (g + n_wg * 4 < p.groups) fetch_past(g + n_wg * 4);
        }
        if (R > 1 && (MORE ? row0 < a.gated : a.gated)) {
            if (l == 0)
#pragma unroll
                for (int r = 0; r + 1 < R; r += 2) {
                    const int row = row0 + r;  // (even, and so is the number of rows in pairs, in whole groups)
                    if (row >= a.rows) continue;
                    const float b0 = a.bias ? a.bias[row] : 0.f, b1 = a.bias ? a.bias[row + 1] : 0.f;
                    a.y[(size_t)b * a.y_batch + (row >> 1)] = activate(acc[r] + b0, a.act0) * (acc[r + 1] + b1);
                }
        } else if (l == 0) {
#pragma unroll
            for (int r = 0; r < R; ++r) {
                const int row = row0 + r, ch = row - e.conv_from;
                if (row >= a.rows) continue;
                float v = acc[r];
                if (a.bias && (!conv || ch < 0 || ch >= e.channels)) v += a.bias[row];
                const int act = MORE && row >= e.act2_from ? e.act2 : row < a.act_split ? a.act0 : a.act1;
                v = MORE ? activate(v, act, e.act_a, e.act_b) : activate(v, act);
                if (mul) v *= bf2f(e.mul[(size_t)min(max(e.mul_tokens[mul_at], 0), e.mul_rows - 1) * e.ld_mul + row]);
                a.y[(size_t)b * a.y_batch + row - (MORE ? a.gated >> 1 : 0)] = v;
                if (a.best_val) {
                    const float t = v != v ? -INFINITY : v;
                    if (t > bv || (t == bv && row < bi)) {
                        bv = t;
                        bi = row;
                    }
                }
            }
        }
    }
    if (a.best_val) {
        // one candidate per row group of lanes, then per wave
#pragma unroll
        for (int off = 32; off >= LPR; off >>= 1) {
            const float ov = __shfl_xor(bv, off, 64);
            const int oi = __shfl_xor(bi, off, 64);
            if (ov > bv || (ov == bv && oi < bi)) {
                bv = ov;
                bi = oi;
            }
        }
        if (lane == 0) {
            wbv[wave] = bv;
            wbi[wave] = bi;
        }
        __syncthreads();
        if (tid == 0) {
            for (int i = 1; i < 4; ++i)
                if (wbv[i] > bv || (wbv[i] == bv && wbi[i] < bi)) {
                    bv = wbv[i];
                    bi = wbi[i];
                }
            a.best_val[blockIdx.x] = bv;
            a.best_idx[blockIdx.x] = bi;
        }
    }
}

template <int LPR, int R, bool MORE>
static void gemv_go(int u, const GemvK &k, dim3 grid, hipStream_t s) {
    const size_t lds = (size_t)k.kp * 4;
    void (*fn)(GemvK) = u == 1 ? k_dense_gemv<LPR, R, 1, MORE> : u == 2 ? k_dense_gemv<LPR, R, 2, MORE> : u == 3 ? k_dense_gemv<LPR, R, 3, MORE>
                      : u == 4 ? k_dense_gemv<LPR, R, 4, MORE> : k_dense_gemv<LPR, R, 5, MORE>;
    if (lds > 65536) (void)hipFuncSetAttribute(reinterpret_cast<const void *>(fn), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
    hipLaunchKernelGGL(fn, grid, dim3(256), lds, s, k);
}

template <int LPR, int R>
static void gemv_pick_u(int u, const GemvK &k, dim3 grid, hipStream_t s) {
    const GemvArgs &a = k.a;
    const bool pairs = a.gated && a.gated < a.rows;
    if (a.in.y_gate || pairs || a.more.conv || a.more.mul || a.more.act2_from < a.rows || a.act0 == BITNET_HIP_ACT_XIELU || a.act1 == BITNET_HIP_ACT_XIELU)
        gemv_go<LPR, R, true>(u, k, grid, s);
    else
        gemv_go<LPR, R, false>(u, k, grid, s);
}

hipError_t launch_dense_gemv(const GemvArgs &a, int *n_wg_out, hipStream_t s) {
    GemvK k;
    k.a = a;
    k.a.latent = nullptr;
    if (a.act_split == 0) k.a.act_split = a.rows;
    if (k.a.in.mean_n == 0) k.a.in.mean_n = a.in.n;
    const int lpr = a.cols <= 64 ? 8 : a.cols <= 256 ? 16 : 64;
    const int chunks = (a.cols + lpr * 8 - 1) / (lpr * 8);
    int u = chunks < 5 ? chunks : 5;
    if (chunks > 5)
        for (int c = 4; c >= 3; --c)
            if ((chunks + c - 1) / c * c < (chunks + u - 1) / u * u) u = c;
    const int step = lpr * 8 * u;
    k.kp = (a.cols + step - 1) / step * step;
    if ((size_t)k.kp * 4 > 150 * 1024) return hipErrorInvalidValue;
    // rows per lane group: enough workgroups to reach every CU twice, then more rows in flight per wave
    const int per = 64 / lpr;
    auto wgs = [&](int r) { return ((long)a.rows + 4l * per * r - 1) / (4l * per * r) * a.batch; };
    int r = 1;
    if (wgs(4) >= 1024) r = 4;
    else if (wgs(2) >= 512 || a.gated) r = 2;
    k.groups = (a.rows + per * r - 1) / (per * r);
    int n_wg = (k.groups + 3) / 4;
    const int cap = 768;  // three workgroups per CU: each forms the whole input again (measured: 512 and 1024 are slower)
    if (a.batch == 1 && n_wg > cap) {
        const int rounds = (n_wg + cap - 1) / cap;
        n_wg = (n_wg + rounds - 1) / rounds;
    }
    if (n_wg_out) *n_wg_out = n_wg;
    k.lat_wg = a.latent ? n_wg : -1;
    if (a.latent) k.lat = *a.latent;
    const dim3 grid(n_wg + (a.latent ? 1 : 0), a.batch);
    if (lpr == 8)
        r == 4 ? gemv_pick_u<8, 4>(u, k, grid, s) : r == 2 ? gemv_pick_u<8, 2>(u, k, grid, s) : gemv_pick_u<8, 1>(u, k, grid, s);
    else if (lpr == 16)
        r == 4 ? gemv_pick_u<16, 4>(u, k, grid, s) : r == 2 ? gemv_pick_u<16, 2>(u, k, grid, s) : gemv_pick_u<16, 1>(u, k, grid, s);
    else
        r == 4 ? gemv_pick_u<64, 4>(u, k, grid, s) : r == 2 ? gemv_pick_u<64, 2>(u, k, grid, s) : gemv_pick_u<64, 1>(u, k, grid, s);
    return hipGetLastError();
}

// ---- many-row matmul --------------------------------------------------------------------------------------------------
// C[m][n] = act(A[m][k] . W[n][k]^T + bias).  Workgroup tile TN x TM in WN x WM waves, K steps of 64 columns staged in LDS by LDS-DMA,
// ST buffers.  256 x 256 in eight waves of 128 x 64 where the launch has the tiles for it (half the bytes per
// product of 128 x 128, and a fragment read from LDS feeds four to eight MFMAs), 128 x 128, and 64 x 64 with four buffers for launches
// that do not fill the chip and would wait for memory at every step.  LDS image of a row: eight 16-byte units, unit q stored at
// q ^ ((row >> 1) & 7) (activations) or q ^ weight_key(row) (weights): the sixteen rows of a ds_read_b128 cover all 64 banks once.  The
// MFMA's A operand is the weight tile (rows = output columns n), its B operand the activation tile; for bf16
// outputs row r of weight fragment i is column 4 FN (r / 4) + 4 i + r % 4 of the wave's tile, so that a lane ends up with 4 FN consecutive
// columns of one output row (stores of 32-byte pieces cost more than the arithmetic of a short product); f32 outputs keep 16 i + r, four
// lanes of 16 bytes side by side.
constexpr int kTileK = 64;

// 64 lanes x 16 bytes from (scalar base + lane offset) to LDS bytes [lds_dst, lds_dst + 1024); invisible to hipcc's vmcnt bookkeeping
__device__ __forceinline__ void dma1k(unsigned lane_off, const void *sbase, unsigned lds_dst) {
    unsigned keep;
    asm volatile("s_mov_b32 %0, m0\n\ts_mov_b32 m0, %3\n\ts_nop 0\n\tglobal_load_lds_dwordx4 %1, %2\n\ts_mov_b32 m0, %0"
                 : "=&s"(keep)
                 : "v"(lane_off), "s"(sbase), "s"(lds_dst)
                 : "memory");
}

template <int FN, bool CF32>
__device__ __forceinline__ int weight_key(int row) {
    return CF32 ? (row >> 1) & 7 : ((row / (4 * FN)) & 3) * 2 + ((row >> 1) & 1);
}

// GROUPED: the row tiles come from a device list, (matrix, first row, rows) each; a matrix's tiles follow one another.
// GATED (bf16 outputs): columns 2 i and 2 i + 1 make column i of the output.
// MUL (bf16 outputs): row i of the output is multiplied by a table's row, the one of its token.
template <int TN, int TM, int WN, int WM, int ST, bool CF32, bool GROUPED = false, bool GATED = false, bool MUL = false>
__global__ __launch_bounds__(64 * WN * WM, 2) void k_dense_gemm(GemmArgsD p, int tiles_n, int tiles_m, int swizzle) {
    extern __shared__ __attribute__((aligned(1024))) uint8_t lds[];
    constexpr int NW = WN * WM, DN = TN / NW / 8, DM = TM / NW / 8;  // DMA instructions per wave and step (eight rows each)
    constexpr int FN = TN / WN / 16, FM = TM / WM / 16;              // 16-row fragments per wave
    constexpr unsigned ABUF = TM * 128, BUF = ABUF + TN * 128;
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    // workgroup -> tile: consecutive workgroups land on the eight XCDs in turn; give each XCD a contiguous run of tiles, and walk
    // the tiles in groups of eight row tiles so that what runs together shares both operands in the XCD's L2
    int id = blockIdx.x;
    int m0, n0, m_end;
    const uint16_t *A = (const uint16_t *)p.a + (size_t)blockIdx.y * p.a_batch;
    const uint16_t *W = p.w + (size_t)blockIdx.y * p.w_batch;
    if (GROUPED) {
        const int total = *p.n_tiles * tiles_n, per = (total + 7) >> 3;
        if ((id >> 3) >= per) return;
        id = (id & 7) * per + (id >> 3);
        if (id >= total) return;
        const int4 tile = p.tiles[id / tiles_n];
        m0 = tile.y, m_end = tile.y + tile.z, n0 = id % tiles_n * TN;
        W += (size_t)tile.x * p.w_batch;
    } else {
        const int total = tiles_n * tiles_m;
        if (swizzle) id = (id & 7) * (total >> 3) + (id >> 3);
        const int gm = 8;
        const int group = id / (gm * tiles_n), first = group * gm, size = tiles_m - first < gm ? tiles_m - first : gm;
        const int tm = first + (id % (gm * tiles_n)) % size, tn = (id % (gm * tiles_n)) / size;
        m0 = tm * TM, n0 = tn * TN, m_end = p.m;
    }
    const int drow = lane >> 3;
    // (lane offsets from the tile's first row: a tile spans less than 4 GiB; rows past the end read the tile's own rows over again)
    const unsigned rows_m = min(TM, m_end - m0), rows_n = min(TN, p.n - n0);
    const bool gathered = GROUPED && p.gather;
    const uint16_t *A0 = gathered ? A : A + (size_t)m0 * p.lda, *W0 = W + (size_t)n0 * p.ldw;
    unsigned oa[DM], ow[DN];
#pragma unroll
    for (int i = 0; i < DM; ++i) {
        const int r = wave * (TM / NW) + i * 8 + drow, unit = (lane & 7) ^ ((r >> 1) & 7);
        const unsigned row = gathered ? (unsigned)p.gather[m0 + (unsigned)r % rows_m] : (unsigned)r % rows_m;
        oa[i] = (unsigned)(row * p.lda + unit * 8) * 2;
    }
#pragma unroll
    for (int i = 0; i < DN; ++i) {
        const int r = wave * (TN / NW) + i * 8 + drow, unit = (lane & 7) ^ weight_key<FN, CF32>(r);
        ow[i] = (unsigned)((unsigned)r % rows_n * p.ldw + unit * 8) * 2;
    }
    const unsigned base = (unsigned)(uintptr_t)(__attribute__((address_space(3))) uint8_t *)lds;
    auto stage = [&](int t) {
        const unsigned dst = base + (t % ST) * BUF;
#pragma unroll
        for (int i = 0; i < DM; ++i) dma1k(oa[i], A0 + t * kTileK, dst + wave * (TM / NW) * 128 + i * 1024);
#pragma unroll
        for (int i = 0; i < DN; ++i) dma1k(ow[i], W0 + t * kTileK, dst + ABUF + wave * (TN / NW) * 128 + i * 1024);
    };
    const int wn = (wave % WN) * (TN / WN), wm = (wave / WN) * (TM / WM);
    const int r16 = lane & 15, g = lane >> 4, sw = (r16 >> 1) & 7;
    constexpr int FS = CF32 ? 16 : 4;  // columns between fragments; neither step changes a row's key: one for all fragments
    const int wr = CF32 ? wn + r16 : wn + (r16 >> 2) * 4 * FN + (r16 & 3);
    f32x4 acc[FN][FM];
#pragma unroll
    for (int i = 0; i < FN; ++i)
#pragma unroll
        for (int j = 0; j < FM; ++j) acc[i][j] = f32x4{0.f, 0.f, 0.f, 0.f};
    const int steps = p.k / kTileK;
    // Fragments are read half a step (32 columns) ahead of the MFMAs that use them, reads and MFMAs interleaved: the middle of a step
    // waits for the next tile, and the barrier there also says that every wave has left the tile whose buffer is requested next.
    bf16x8 fa[2][FM], fw[2][FN];
    auto read = [&](int t, int kk) {
        const uint8_t *la = lds + (t % ST) * BUF, *lw = la + ABUF;
        const int q = ((kk * 4 + g) ^ sw) * 16, qw = ((kk * 4 + g) ^ weight_key<FN, CF32>(wr)) * 16;
#pragma unroll
        for (int j = 0; j < FM; ++j) fa[kk][j] = *reinterpret_cast<const bf16x8 *>(la + (wm + j * 16 + r16) * 128 + q);
#pragma unroll
        for (int i = 0; i < FN; ++i) fw[kk][i] = *reinterpret_cast<const bf16x8 *>(lw + (wr + i * FS) * 128 + qw);
    };
    auto multiply = [&](int kk) {
#pragma unroll
        for (int i = 0; i < FN; ++i)
#pragma unroll
            for (int j = 0; j < FM; ++j) acc[i][j] = mfma_bf16(fw[kk][i], fa[kk][j], acc[i][j]);
#pragma unroll
        for (int i = 0; i < (FN + FM) / 2; ++i) {
            __builtin_amdgcn_sched_group_barrier(0x100, 2, 0);                         // two LDS reads
            __builtin_amdgcn_sched_group_barrier(0x008, 2 * FN * FM / (FN + FM), 0);  // their share of the MFMAs
        }
    };
#pragma unroll
    for (int t = 0; t < ST; ++t)
        if (t < steps) stage(t);
    // (loads return in order: a tile is there once at most the later ones are outstanding)
    if (steps >= ST)
        asm volatile("s_waitcnt vmcnt(%0)" ::"n"((ST - 1) * (DM + DN)) : "memory");
    else
        asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
    __syncthreads();
    read(0, 0);
    for (int t = 0; t < steps; ++t) {
        read(t, 1);
        multiply(0);
        if (t + ST - 1 < steps)
            asm volatile("s_waitcnt vmcnt(%0) lgkmcnt(0)" ::"n"((ST - 2) * (DM + DN)) : "memory");
        else
            asm volatile("s_waitcnt vmcnt(0) lgkmcnt(0)" ::: "memory");
        __syncthreads();
        if (t + ST < steps) stage(t + ST);
        read(t + 1, 0);  // (behind the last step: bytes nobody uses)
        multiply(1);
    }
    // this lane's columns: nl + i * FS + e
    const int nl = n0 + wn + g * (CF32 ? 4 : 4 * FN), nlast = nl + (FN - 1) * FS + 3;
    const bool vec = (p.ldc & 7) == 0 && (p.c_batch & 7) == 0 && ((uintptr_t)p.c & 15) == 0;
    // the activation: one for the whole wave unless the split runs through its columns
    const int mine = nlast < p.act_split ? p.act0 : nl >= p.act_split ? p.act1 : -1, act0 = __builtin_amdgcn_readfirstlane(mine);
    const int act = __all(mine == act0) ? act0 : -1;
#pragma unroll
    for (int j = 0; j < FM; ++j) {
        const int m = m0 + wm + j * 16 + r16;
        if (m >= m_end) continue;
        const size_t o = (size_t)blockIdx.y * p.c_batch + (size_t)m * p.ldc + nl;
        if (p.bias)
#pragma unroll
            for (int i = 0; i < FN; ++i)
#pragma unroll
                for (int e = 0; e < 4; ++e) acc[i][j][e] += p.bias[min(nl + i * FS + e, p.n - 1)];
        if (GATED) {
            float r[2 * FN];
#pragma unroll
            for (int i = 0; i < FN; ++i)
#pragma unroll
                for (int e = 0; e < 4; e += 2) {
                    const float v = acc[i][j][e], z = p.act0 == BITNET_HIP_ACT_GELU_TANH ? 2.0f * gelu_argument(v) : v;
                    const float sg = __builtin_amdgcn_rcpf(1.0f + __expf(-z));
                    r[2 * i + e / 2] = (p.act0 == BITNET_HIP_ACT_SILU || p.act0 == BITNET_HIP_ACT_GELU_TANH ? v * sg : activate(v, p.act0)) * acc[i][j][e + 1];
                }
            uint16_t *dst = (uint16_t *)p.c + (size_t)blockIdx.y * p.c_batch + (size_t)m * p.ldc + nl / 2;
#pragma unroll
            for (int i = 0; i < 2 * FN; i += 4) {
                if (vec && nl + 2 * i + 7 < p.n) {
                    *reinterpret_cast<bf16x4 *>(dst + i) = bf16x4{(__bf16)r[i], (__bf16)r[i + 1], (__bf16)r[i + 2], (__bf16)r[i + 3]};
                } else {
#pragma unroll
                    for (int e = 0; e < 4; ++e)
                        if (nl + 2 * (i + e) < p.n) dst[i + e] = f2bf(r[i + e]);
                }
            }
            continue;
        }
        auto apply = [&](auto f) {
#pragma unroll
            for (int i = 0; i < FN; ++i)
#pragma unroll
                for (int e = 0; e < 4; ++e) acc[i][j][e] = f(acc[i][j][e], nl + i * FS + e);
        };
        // (exp(v) - 1 loses what a bf16 output does not keep)
        auto xielu = [&](float v) { return 0.5f * v + (v > 0.f ? p.more.act_a * v * v : p.more.act_b * (__expf(v) - 1.0f - v)); };
        if (act < 0)
            apply([&](float v, int n) {
                const int f = n < p.act_split ? p.act0 : p.act1;
                const float sg = __builtin_amdgcn_rcpf(1.0f + __expf(-v)), r = fmaxf(v, 0.0f);
                return f == BITNET_HIP_ACT_SILU ? v * sg : f == BITNET_HIP_ACT_SIGMOID ? sg : f == BITNET_HIP_ACT_RELU2 ? r * r : f == BITNET_HIP_ACT_XIELU ? xielu(v) : activate(v, f);
            });
        else if (act == BITNET_HIP_ACT_SILU)
            apply([](float v, int) { return v * __builtin_amdgcn_rcpf(1.0f + __expf(-v)); });
        else if (act == BITNET_HIP_ACT_SIGMOID)
            apply([](float v, int) { return __builtin_amdgcn_rcpf(1.0f + __expf(-v)); });
        else if (act == BITNET_HIP_ACT_RELU2)
            apply([](float v, int) { return activate(v, BITNET_HIP_ACT_RELU2); });
        else if (act == BITNET_HIP_ACT_GELU_TANH)
            apply([](float v, int) { return v * __builtin_amdgcn_rcpf(1.0f + __expf(-2.0f * gelu_argument(v))); });
        else if (act == BITNET_HIP_ACT_XIELU)
            apply([&](float v, int) { return xielu(v); });
        if (MUL) {
            const int token = min(max(p.more.mul_tokens[*p.more.mul_at + m], 0), p.more.mul_rows - 1);
            const uint16_t *mul = p.more.mul + (size_t)token * p.more.ld_mul;
            apply([&](float v, int n) { return v * bf2f(mul[min(n, p.n - 1)]); });
        }
        if (CF32) {
#pragma unroll
            for (int i = 0; i < FN; ++i) {
                float *dst = (float *)p.c + o + i * FS;
                if (vec && nl + i * FS + 3 < p.n) {
                    *reinterpret_cast<f32x4 *>(dst) = acc[i][j];
                } else {
#pragma unroll
                    for (int e = 0; e < 4; ++e)
                        if (nl + i * FS + e < p.n) dst[e] = acc[i][j][e];
                }
            }
        } else {
#pragma unroll
            for (int i = 0; i < FN; i += 2) {
                uint16_t *dst = (uint16_t *)p.c + o + i * FS;
                if (vec && nl + i * FS + 7 < p.n) {
                    *reinterpret_cast<bf16x8 *>(dst) =
                        bf16x8{(__bf16)acc[i][j][0],     (__bf16)acc[i][j][1],     (__bf16)acc[i][j][2],     (__bf16)acc[i][j][3],
                               (__bf16)acc[i + 1][j][0], (__bf16)acc[i + 1][j][1], (__bf16)acc[i + 1][j][2], (__bf16)acc[i + 1][j][3]};
                } else {
#pragma unroll
                    for (int e = 0; e < 8; ++e)
                        if (nl + i * FS + e < p.n) dst[e] = f2bf(acc[i + (e >> 2)][j][e & 3]);
                }
            }
        }
    }
}

template <int T, int ST>
static hipError_t grouped_go(const GemmArgsD &a, hipStream_t s) {
    const int tn = (a.n + T - 1) / T;
    constexpr size_t lds = (size_t)ST * T * 256;
    auto fn = a.gated ? k_dense_gemm<T, T, 2, 2, ST, false, true, true> : k_dense_gemm<T, T, 2, 2, ST, false, true>;
    if (lds > 65536) {
        const hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void *>(fn), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
        if (e != hipSuccess) return e;
    }
    hipLaunchKernelGGL(fn, dim3((tn * a.max_tiles + 7) / 8 * 8), dim3(256), lds, s, a, tn, 0, 0);
    return hipGetLastError();
}

template <int T, int WN, int WM, int ST, bool MUL = false>
static hipError_t gemm_go(const GemmArgsD &a, hipStream_t s) {
    const int tn = (a.n + T - 1) / T, tm = (a.m + T - 1) / T, swz = (tn * tm) % 8 == 0 ? 1 : 0;
    constexpr size_t lds = (size_t)ST * T * 256;
    auto fn = MUL       ? k_dense_gemm<T, T, WN, WM, ST, false, false, false, MUL>
              : a.gated ? k_dense_gemm<T, T, WN, WM, ST, false, false, true>
              : a.c_f32 ? k_dense_gemm<T, T, WN, WM, ST, true>
                        : k_dense_gemm<T, T, WN, WM, ST, false>;
    if (lds > 65536) {
        const hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void *>(fn), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
        if (e != hipSuccess) return e;
    }
    hipLaunchKernelGGL(fn, dim3(tn * tm, a.batch), dim3(64 * WN * WM), lds, s, a, tn, tm, swz);
    return hipGetLastError();
}

// f32 activations: f32 multiply-adds on a 64 x 64 tile, 4 x 4 per thread
template <bool GROUPED>
__global__ __launch_bounds__(256) void k_dense_gemm_f32(GemmArgsD p) {
    __shared__ float sa[16][68], sw[16][68];
    const int tid = threadIdx.x, tx = tid & 15, ty = tid >> 4;
    int m0 = blockIdx.y * 64, m_end = p.m;
    const int n0 = blockIdx.x * 64;
    const float *A = (const float *)p.a + (size_t)blockIdx.z * p.a_batch;
    const uint16_t *W = p.w + (size_t)blockIdx.z * p.w_batch;
    if (GROUPED) {
        if ((int)blockIdx.y >= *p.n_tiles) return;
        const int4 tile = p.tiles[blockIdx.y];
        m0 = tile.y, m_end = tile.y + tile.z;
        W += (size_t)tile.x * p.w_batch;
    }
    float acc[4][4] = {};
    const int lr = tid >> 2, lk = (tid & 3) * 4;
    int ar = m0 + lr < m_end ? m0 + lr : m_end - 1;
    if (GROUPED && p.gather) ar = p.gather[ar];
    const int wr = n0 + lr < p.n ? n0 + lr : p.n - 1;
    for (int k0 = 0; k0 < p.k; k0 += 16) {
        const f32x4 av = *reinterpret_cast<const f32x4 *>(A + (size_t)ar * p.lda + k0 + lk);
        const u32x2 wv = *reinterpret_cast<const u32x2 *>(W + (size_t)wr * p.ldw + k0 + lk);
        __syncthreads();
        sa[lk][lr] = av.x, sa[lk + 1][lr] = av.y, sa[lk + 2][lr] = av.z, sa[lk + 3][lr] = av.w;
        sw[lk][lr] = bf2f(wv.x & 0xffffu), sw[lk + 1][lr] = bf2f(wv.x >> 16), sw[lk + 2][lr] = bf2f(wv.y & 0xffffu), sw[lk + 3][lr] = bf2f(wv.y >> 16);
        __syncthreads();
#pragma unroll
        for (int k = 0; k < 16; ++k) {
            float x[4], w[4];
#pragma unroll
            for (int i = 0; i < 4; ++i) x[i] = sa[k][ty * 4 + i], w[i] = sw[k][tx * 4 + i];
#pragma unroll
            for (int i = 0; i < 4; ++i)
#pragma unroll
                for (int j = 0; j < 4; ++j) acc[i][j] = fmaf(x[i], w[j], acc[i][j]);
        }
    }
    for (int i = 0; i < 4; ++i) {
        const int m = m0 + ty * 4 + i;
        if (m >= m_end) break;
        for (int j = 0; j < 4; ++j) {
            const int n = n0 + tx * 4 + j;
            if (n >= p.n) break;
            if (p.gated && (j & 1)) continue;
            float v = activate(acc[i][j] + (p.bias ? p.bias[n] : 0.f), n < p.act_split ? p.act0 : p.act1, p.more.act_a, p.more.act_b);
            if (p.more.mul) v *= bf2f(p.more.mul[(size_t)min(max(p.more.mul_tokens[*p.more.mul_at + m], 0), p.more.mul_rows - 1) * p.more.ld_mul + n]);
            size_t o = (size_t)blockIdx.z * p.c_batch + (size_t)m * p.ldc + n;
            if (p.gated) {  // (n is even here, and so is the number of columns)
                v *= acc[i][j < 3 ? j + 1 : 3] + (p.bias ? p.bias[n + 1] : 0.f);
                o -= n / 2;
            }
            if (p.c_f32)
                ((float *)p.c)[o] = v;
            else
                ((uint16_t *)p.c)[o] = f2bf(v);
        }
    }
}

hipError_t launch_dense_gemm(const GemmArgsD &args, hipStream_t s) {
    GemmArgsD a = args;
    if (a.m <= 0 || a.n <= 0) return hipSuccess;
    if (a.act_split == 0) a.act_split = a.n;
    if (a.gated && !a.a_f32 && a.c_f32) return hipErrorInvalidValue;
    if (a.tiles) {
        if (a.a_f32) {
            if (a.tile != 64) return hipErrorInvalidValue;
            hipLaunchKernelGGL(k_dense_gemm_f32<true>, dim3((a.n + 63) / 64, a.max_tiles, 1), dim3(256), 0, s, a);
            return hipGetLastError();
        }
        if (a.c_f32) return hipErrorInvalidValue;
        return a.tile == 128 ? grouped_go<128, 2>(a, s) : a.tile == 64 ? grouped_go<64, 4>(a, s) : hipErrorInvalidValue;
    }
    if (a.a_f32) {
        hipLaunchKernelGGL(k_dense_gemm_f32<false>, dim3((a.n + 63) / 64, (a.m + 63) / 64, a.batch), dim3(256), 0, s, a);
        return hipGetLastError();
    }
    if (a.more.mul) return a.c_f32 || a.gated ? hipErrorInvalidValue : gemm_go<64, 2, 2, 4, true>(a, s);
    auto tiles = [&](int t) { return (long)((a.n + t - 1) / t) * ((a.m + t - 1) / t) * a.batch; };
    if (a.k <= 1024 && tiles(64) >= 1024) return gemm_go<64, 2, 2, 2>(a, s);  // few steps: what counts is how many workgroups overlap their ends
    if (tiles(128) >= 200) {
        // measured per K step: 2.05 us for a round of 256 large tiles (one per CU), 1.15 us for a round of 512 of the others (two per CU);
        // a column tile of the large kind that sticks out over the last column costs a third more
        const double large = (a.n % 256 ? 2.7 : 2.05) * ((tiles(256) + 255) / 256), small = 1.15 * ((tiles(128) + 511) / 512);
        return large <= small ? gemm_go<256, 2, 4, 2>(a, s) : gemm_go<128, 2, 2, 2>(a, s);
    }
    return gemm_go<64, 2, 2, 4>(a, s);
}

}  // namespace bitnet_hip
