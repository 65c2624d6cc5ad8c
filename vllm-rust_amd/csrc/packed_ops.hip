// Kernels that every packed-step executor needs around its mixers and linears: RMS and layer norm of the f32 residual stream (a
// gain per column or one gain for the row), the norms around a residual sum in one pass, gated activations, the inverse
// map and the weighted combine of a mixture of experts whose (token, slot) pairs were sorted into expert blocks, greedy ids of f32
// logits rows, a fill, the step table of a rotary position code.
#include "vmx_kernels.h"
#include <float.h>
#include <math.h>
#include <algorithm>

namespace {

// out[r] = x[rows ? rows[r] : r] / sqrt(mean(x^2) + eps) * w, f32 statistics; out in f32 or bf16; w one gain per column or
// (w_scalar) a single gain for the whole row.  CENTERED: the row's mean is taken off first (layer norm; the statistic is then the
// variance).  Rows up to 4096 wide stay in registers between the statistics and the scaling (one trip to memory), wider rows are
// read once per pass.
template <bool CENTERED>
__global__ __launch_bounds__(256) void row_norm_f32in_kernel(void *__restrict__ out, int out_f32, const float *__restrict__ x,
                                                              const int32_t *__restrict__ rows, const uint16_t *__restrict__ w, int w_scalar,
                                                              int width, float eps) {
    __shared__ float red[4];
    const int r = blockIdx.x;
    const float *src = x + (int64_t)(rows ? rows[r] : r) * width;
    constexpr int PT = 16;
    float xv[PT], wv[PT];
    const bool held = width <= 256 * PT;
    float ss = 0.f, mean = 0.f;
    if (held) {
#pragma unroll
        for (int u = 0; u < PT; u++) {
            const int i = threadIdx.x + 256 * u;
            xv[u] = i < width ? src[i] : 0.f;
            wv[u] = i < width ? vmx_bf16_to_f32(w[w_scalar ? 0 : i]) : 0.f;
        }
        if constexpr (CENTERED) {
            float s = 0.f;
#pragma unroll
            for (int u = 0; u < PT; u++) s += xv[u];
            mean = vmx_block_sum_256(s, red) / (float)width;
#pragma unroll
            for (int u = 0; u < PT; u++) xv[u] = threadIdx.x + 256 * u < width ? xv[u] - mean : 0.f;
        }
#pragma unroll
        for (int u = 0; u < PT; u++) ss += xv[u] * xv[u];   // same order as the strided loop below
    } else {
        if constexpr (CENTERED) {
            float s = 0.f;
            for (int i = threadIdx.x; i < width; i += 256) s += src[i];
            mean = vmx_block_sum_256(s, red) / (float)width;
        }
        for (int i = threadIdx.x; i < width; i += 256) ss += (src[i] - mean) * (src[i] - mean);
    }
    ss = vmx_block_sum_256(ss, red);
    const float inv = 1.0f / sqrtf(ss / (float)width + eps);
    if (held) {
#pragma unroll
        for (int u = 0; u < PT; u++) {
            const int i = threadIdx.x + 256 * u;
            if (i < width) {
                const float v = xv[u] * inv * wv[u];
                if (out_f32) ((float *)out)[(int64_t)r * width + i] = v;
                else ((uint16_t *)out)[(int64_t)r * width + i] = vmx_f32_to_bf16(v);
            }
        }
        return;
    }
    for (int i = threadIdx.x; i < width; i += 256) {
        const float v = (src[i] - mean) * inv * vmx_bf16_to_f32(w[w_scalar ? 0 : i]);
        if (out_f32) ((float *)out)[(int64_t)r * width + i] = v;
        else ((uint16_t *)out)[(int64_t)r * width + i] = vmx_f32_to_bf16(v);
    }
}

// The norms around a residual sum in one pass over the row: x <- [x +] post_mul * N(y) * w_post (w_post NULL: y itself), h = N(x) * w_next
// (w_next NULL: h = x, or no h).  y[t] is a row of numbers, a row of the embedding table, the combined result of a mixture of experts,
// or (SIDE) the scaled sum of two branches that each have a norm of their own.  N as above, centred or not.  A thread keeps HELD groups of VEC neighbouring columns in registers from the first read to the last store, and every load
// that does not depend on a statistic is issued before the first one.  HELD 0: any width, y is formed anew in every pass (at most
// three, five with two branches) and the new x is read back by the thread that wrote it.
template <int VEC> struct SandwichVec;
template <> struct SandwichVec<4> {
    static __device__ __forceinline__ void ld(const float *p, float *v) {
        const float4 f = *reinterpret_cast<const float4 *>(p);
        v[0] = f.x, v[1] = f.y, v[2] = f.z, v[3] = f.w;
    }
    static __device__ __forceinline__ void ld(const uint16_t *p, float *v) {
        const uint2 u = *reinterpret_cast<const uint2 *>(p);
        v[0] = vmx_bf16_to_f32((uint16_t)u.x), v[1] = vmx_bf16_to_f32((uint16_t)(u.x >> 16));
        v[2] = vmx_bf16_to_f32((uint16_t)u.y), v[3] = vmx_bf16_to_f32((uint16_t)(u.y >> 16));
    }
    static __device__ __forceinline__ void st(float *p, const float *v) { *reinterpret_cast<float4 *>(p) = make_float4(v[0], v[1], v[2], v[3]); }
    static __device__ __forceinline__ void st(uint16_t *p, const float *v) {
        *reinterpret_cast<uint2 *>(p) = make_uint2((uint32_t)vmx_f32_to_bf16(v[0]) | ((uint32_t)vmx_f32_to_bf16(v[1]) << 16),
                                                   (uint32_t)vmx_f32_to_bf16(v[2]) | ((uint32_t)vmx_f32_to_bf16(v[3]) << 16));
    }
};
template <> struct SandwichVec<1> {
    static __device__ __forceinline__ void ld(const float *p, float *v) { v[0] = p[0]; }
    static __device__ __forceinline__ void ld(const uint16_t *p, float *v) { v[0] = vmx_bf16_to_f32(p[0]); }
    static __device__ __forceinline__ void st(float *p, const float *v) { p[0] = v[0]; }
    static __device__ __forceinline__ void st(uint16_t *p, const float *v) { p[0] = vmx_f32_to_bf16(v[0]); }
};

template <int HELD, int VEC, bool SIDE>
__global__ __launch_bounds__(256) void sandwich_norm_kernel(const VmxSandwich a) {
    using V = SandwichVec<VEC>;
    __shared__ float red[8][4];      // a row per reduction: one barrier each
    constexpr int G = HELD ? HELD : 1;
    const int t = blockIdx.x, tid = threadIdx.x, W = a.width;
    float *x = a.x + (int64_t)t * W;
    const float inv_w = 1.0f / (float)W;
    auto block_sum = [&](float v, int k) {
        v = vmx_wave_sum(v);
        if ((tid & 63) == 0) red[k][tid >> 6] = v;
        __syncthreads();
        return (red[k][0] + red[k][1]) + (red[k][2] + red[k][3]);
    };
    const float sg = a.shared_gate ? 1.0f / (1.0f + expf(-a.shared_gate[(int64_t)t * a.ld_shared_gate])) : 1.0f;
    const uint16_t *erow = nullptr;
    if (a.embed) {
        const int id = a.tokens[t];
        erow = a.embed + (int64_t)(id < 0 ? 0 : (id >= a.vocab ? a.vocab - 1 : id)) * W;
    }
    if constexpr (HELD > 0) {
        float y[G][VEC], xv[G][VEC], wp[G][VEC], wn[G][VEC];
        float sd[SIDE ? G : 1][VEC], wy[SIDE ? G : 1][VEC], ws[SIDE ? G : 1][VEC];
        int col[G];
        bool in[G];
#pragma unroll
        for (int u = 0; u < G; u++) {
            col[u] = VEC * (tid + 256 * u);
            in[u] = col[u] < W;
#pragma unroll
            for (int e = 0; e < VEC; e++) y[u][e] = xv[u][e] = wp[u][e] = wn[u][e] = 0.f;
            if constexpr (SIDE)
#pragma unroll
                for (int e = 0; e < VEC; e++) sd[u][e] = wy[u][e] = ws[u][e] = 0.f;
        }
#pragma unroll
        for (int u = 0; u < G; u++)
            if (in[u]) {
                if (a.embed) V::ld(erow + col[u], y[u]);
                else if (!a.pair_rows) V::ld(a.y + (int64_t)t * W + col[u], y[u]);
                if (a.accumulate) V::ld(x + col[u], xv[u]);
                if (a.w_post) V::ld(a.w_post + col[u], wp[u]);
                if constexpr (SIDE) {
                    V::ld(a.side + (int64_t)t * W + col[u], sd[u]);
                    V::ld(a.w_y + col[u], wy[u]);
                    V::ld(a.w_side + col[u], ws[u]);
                }
                if (a.w_next) V::ld(a.w_next + col[u], wn[u]);
            }
        if (a.pair_rows && !a.embed) {
            for (int s0 = 0; s0 < a.top; s0 += 4) {     // four experts' rows in flight
                float w4[4];
                int64_t r4[4];
#pragma unroll
                for (int s = 0; s < 4; s++) {
                    const int64_t p = (int64_t)t * a.top + min(s0 + s, a.top - 1);
                    w4[s] = s0 + s < a.top ? a.pair_w[p] : 0.f;
                    r4[s] = (int64_t)a.pair_rows[p] * W;
                }
#pragma unroll
                for (int u = 0; u < G; u++)
                    if (in[u]) {
                        float v[4][VEC];
#pragma unroll
                        for (int s = 0; s < 4; s++) V::ld(a.y + r4[s] + col[u], v[s]);
#pragma unroll
                        for (int s = 0; s < 4; s++)
#pragma unroll
                            for (int e = 0; e < VEC; e++) y[u][e] = fmaf(w4[s], v[s][e], y[u][e]);
                    }
            }
            if (a.shared)
#pragma unroll
                for (int u = 0; u < G; u++)
                    if (in[u]) {
                        float v[VEC];
                        V::ld(a.shared + (int64_t)t * W + col[u], v);
#pragma unroll
                        for (int e = 0; e < VEC; e++) y[u][e] = fmaf(sg, v[e], y[u][e]);
                    }
        }
        auto statistics = [&](const float (&v)[G][VEC], int k, float &mean) {
            mean = 0.f;
            if (a.centered) {
                float s = 0.f;
#pragma unroll
                for (int u = 0; u < G; u++)
#pragma unroll
                    for (int e = 0; e < VEC; e++) s += v[u][e];     // columns past the row are 0
                mean = block_sum(s, k) * inv_w;
            }
            float ss = 0.f;
#pragma unroll
            for (int u = 0; u < G; u++)
#pragma unroll
                for (int e = 0; e < VEC; e++) {
                    const float d = in[u] ? v[u][e] - mean : 0.f;
                    ss = fmaf(d, d, ss);
                }
            return 1.0f / sqrtf(block_sum(ss, k + 1) * inv_w + a.eps);
        };
        float mean = 0.f, inv = 1.f;
        if constexpr (SIDE) {
            float mean_s;
            const float iy = statistics(y, 4, mean), is = statistics(sd, 6, mean_s);
#pragma unroll
            for (int u = 0; u < G; u++)
#pragma unroll
                for (int e = 0; e < VEC; e++)   // columns past the row have no gains: 0
                    y[u][e] = a.side_mul * ((y[u][e] - mean) * iy * wy[u][e] + (sd[u][e] - mean_s) * is * ws[u][e]);
        }
        if (a.w_post) inv = statistics(y, 0, mean) * a.post_mul;
        else mean = 0.f, inv = a.post_mul;
#pragma unroll
        for (int u = 0; u < G; u++) {
#pragma unroll
            for (int e = 0; e < VEC; e++) xv[u][e] = in[u] ? xv[u][e] + (y[u][e] - mean) * inv * (a.w_post ? wp[u][e] : 1.f) : 0.f;
            if (in[u]) V::st(x + col[u], xv[u]);
        }
        if (a.copy_h) {
#pragma unroll
            for (int u = 0; u < G; u++)
                if (in[u]) {
                    if (a.h_f32) V::st((float *)a.h + (int64_t)t * W + col[u], xv[u]);
                    else V::st((uint16_t *)a.h + (int64_t)t * W + col[u], xv[u]);
                }
            return;
        }
        if (!a.w_next) return;
        inv = statistics(xv, 2, mean);
#pragma unroll
        for (int u = 0; u < G; u++) {
            if (!in[u]) continue;
#pragma unroll
            for (int e = 0; e < VEC; e++) xv[u][e] = (xv[u][e] - mean) * inv * wn[u][e];
            if (a.h_f32) V::st((float *)a.h + (int64_t)t * W + col[u], xv[u]);
            else V::st((uint16_t *)a.h + (int64_t)t * W + col[u], xv[u]);
        }
    } else {
        auto y_at = [&](int i) {
            if (a.embed) return vmx_bf16_to_f32(erow[i]);
            if (!a.pair_rows) return a.y[(int64_t)t * W + i];
            float v = 0.f;
            for (int s = 0; s < a.top; s++) v = fmaf(a.pair_w[(int64_t)t * a.top + s], a.y[(int64_t)a.pair_rows[(int64_t)t * a.top + s] * W + i], v);
            if (a.shared) v = fmaf(sg, a.shared[(int64_t)t * W + i], v);
            return v;
        };
        auto statistics = [&](auto &&at, int k, float &mean) {
            mean = 0.f;
            if (a.centered) {
                float s = 0.f;
                for (int i = tid; i < W; i += 256) s += at(i);
                mean = block_sum(s, k) * inv_w;
            }
            float ss = 0.f;
            for (int i = tid; i < W; i += 256) {
                const float d = at(i) - mean;
                ss = fmaf(d, d, ss);
            }
            return 1.0f / sqrtf(block_sum(ss, k + 1) * inv_w + a.eps);
        };
        float mean_y = 0.f, mean_s = 0.f, iy = 1.f, is = 1.f;
        if constexpr (SIDE) {
            iy = statistics(y_at, 4, mean_y);
            is = statistics([&](int i) { return a.side[(int64_t)t * W + i]; }, 6, mean_s);
        }
        auto branch_at = [&](int i) {   // what goes into the norm after the sublayer
            if constexpr (SIDE)
                return a.side_mul * ((y_at(i) - mean_y) * iy * vmx_bf16_to_f32(a.w_y[i]) +
                                     (a.side[(int64_t)t * W + i] - mean_s) * is * vmx_bf16_to_f32(a.w_side[i]));
            return y_at(i);
        };
        float mean = 0.f, inv = a.post_mul;
        if (a.w_post) inv = statistics(branch_at, 0, mean) * a.post_mul;
        for (int i = tid; i < W; i += 256) {
            const float v = (a.accumulate ? x[i] : 0.f) + (branch_at(i) - mean) * inv * (a.w_post ? vmx_bf16_to_f32(a.w_post[i]) : 1.f);
            x[i] = v;
            if (a.copy_h) {
                if (a.h_f32) ((float *)a.h)[(int64_t)t * W + i] = v;
                else ((uint16_t *)a.h)[(int64_t)t * W + i] = vmx_f32_to_bf16(v);
            }
        }
        if (!a.w_next || a.copy_h) return;
        inv = statistics([&](int i) { return x[i]; }, 2, mean);
        for (int i = tid; i < W; i += 256) {
            const float v = (x[i] - mean) * inv * vmx_bf16_to_f32(a.w_next[i]);
            if (a.h_f32) ((float *)a.h)[(int64_t)t * W + i] = v;
            else ((uint16_t *)a.h)[(int64_t)t * W + i] = vmx_f32_to_bf16(v);
        }
    }
}

// Norm after the sum, over equal consecutive groups of the row: v = acc[t] (w != NULL: every group divided by its own
// sqrt(mean(group^2) + eps), then times w); x[t] = v (f32), h[t] = v (f32 or bf16: what the next products read), acc[t] = alpha * v
// (the sum the next sublayer's result is added to).  One workgroup per row, one group after the other.
__global__ __launch_bounds__(256) void group_norm_post_kernel(float *__restrict__ acc, float *__restrict__ x, void *__restrict__ h, int h_f32,
                                                               const uint16_t *__restrict__ w, int groups, int width, float eps, float alpha) {
    __shared__ float red[4];
    const int64_t row = (int64_t)blockIdx.x * width;
    const int n = width / groups;
    for (int g = 0; g < groups; g++) {
        float inv = 1.0f;
        if (w) {
            float ss = 0.f;
            for (int i = threadIdx.x; i < n; i += 256) {
                const float v = acc[row + g * n + i];
                ss = fmaf(v, v, ss);
            }
            ss = vmx_block_sum_256(ss, red);
            inv = 1.0f / sqrtf(ss / (float)n + eps);
        }
        for (int i = threadIdx.x; i < n; i += 256) {   // a thread rewrites only what it read itself
            const int c = g * n + i;
            float v = acc[row + c] * inv;
            if (w) v *= vmx_bf16_to_f32(w[c]);
            x[row + c] = v;
            if (h_f32) ((float *)h)[row + c] = v;
            else ((uint16_t *)h)[row + c] = vmx_f32_to_bf16(v);
            acc[row + c] = alpha * v;
        }
    }
}

// out[r] = x[rows ? rows[r] : r] normed in groups as above, f32 or bf16 (the rows the output matrix reads)
__global__ __launch_bounds__(256) void group_norm_rows_kernel(void *__restrict__ out, int out_f32, const float *__restrict__ x,
                                                               const int32_t *__restrict__ rows, const uint16_t *__restrict__ w, int groups,
                                                               int width, float eps) {
    __shared__ float red[4];
    const float *src = x + (int64_t)(rows ? rows[blockIdx.x] : blockIdx.x) * width;
    const int64_t row = (int64_t)blockIdx.x * width;
    const int n = width / groups;
    for (int g = 0; g < groups; g++) {
        float ss = 0.f;
        for (int i = threadIdx.x; i < n; i += 256) ss = fmaf(src[g * n + i], src[g * n + i], ss);
        ss = vmx_block_sum_256(ss, red);
        const float inv = 1.0f / sqrtf(ss / (float)n + eps);
        for (int i = threadIdx.x; i < n; i += 256) {
            const int c = g * n + i;
            const float v = src[c] * inv * vmx_bf16_to_f32(w[c]);
            if (out_f32) ((float *)out)[row + c] = v;
            else ((uint16_t *)out)[row + c] = vmx_f32_to_bf16(v);
        }
    }
}

// act[r, j] = silu(s g) * (s u) * sigmoid(out_gate[r]) with g = gu[r, j], u = gu[r, up_off + j]: the gated activation of an expert
// whose INPUT was scaled by s (both products are linear in their input, so the scale is applied to their results), and a
// sigmoid gate per row on what goes into the down projection (linear too).  s = in_w[in_ids ? in_ids[r] : r] (ids outside
// [0, in_limit) are padding rows: 0); in_w NULL: 1; out_gate NULL: none.
__global__ __launch_bounds__(256) void glu_silu_scaled_kernel(void *__restrict__ act, int act_f32, const float *__restrict__ gu, int64_t ldgu,
                                                               int up_off, int ff, const float *__restrict__ in_w,
                                                               const int32_t *__restrict__ in_ids, int in_limit,
                                                               const float *__restrict__ out_gate, int64_t ldgate) {
    const int64_t r = blockIdx.x;
    const int j = blockIdx.y * 256 + threadIdx.x;
    if (j >= ff) return;
    float s = 1.0f;
    if (in_w) {
        const int id = in_ids ? in_ids[r] : (int)r;
        s = (id >= 0 && id < in_limit) ? in_w[id] : 0.f;
    }
    const float g = s * gu[r * ldgu + j], u = s * gu[r * ldgu + up_off + j];
    float v = g / (1.0f + expf(-g)) * u;
    if (out_gate) v *= 1.0f / (1.0f + expf(-out_gate[r * ldgate]));
    if (act_f32) ((float *)act)[r * ff + j] = v;
    else ((uint16_t *)act)[r * ff + j] = vmx_f32_to_bf16(v);
}

// inv[pair] = position of the pair in the expert-sorted list
__global__ __launch_bounds__(256) void moe_inverse_kernel(int32_t *__restrict__ inv, const int32_t *__restrict__ sorted,
                                                           const int32_t *__restrict__ total, int numel) {
    const int i = blockIdx.x * 256 + threadIdx.x;
    if (i < *total) {
        const int p = sorted[i];
        if (p >= 0 && p < numel) inv[p] = i;
    }
}

// x[t] += (sum_slot w[t, slot] * y[inv[t * k + slot]] (slot order) + shared[t]) * sigmoid(gate[t])   (shared, gate optional; w NULL: 1)
__global__ __launch_bounds__(256) void moe_combine_f32_kernel(float *__restrict__ x, const float *__restrict__ y,
                                                               const int32_t *__restrict__ inv, const float *__restrict__ w, int k,
                                                               const float *__restrict__ shared, const float *__restrict__ gate,
                                                               int64_t ldgate, int width) {
    const int t = blockIdx.x, i = blockIdx.y * 256 + threadIdx.x;   // tokens on x (no 65535 limit)
    if (i >= width) return;
    float acc = 0.f;
    for (int s = 0; s < k; s++) acc = fmaf(w ? w[(int64_t)t * k + s] : 1.0f, y[(int64_t)inv[(int64_t)t * k + s] * width + i], acc);
    if (shared) acc += shared[(int64_t)t * width + i];
    if (gate) acc *= 1.0f / (1.0f + expf(-gate[(int64_t)t * ldgate + i]));
    x[(int64_t)t * width + i] += acc;
}

// Greedy ids in two launches: chunk winners as keys (order-preserving value bits | inverted index, so the largest key is the
// largest value with the smallest index), then the winner of a row's keys.
__device__ __forceinline__ unsigned long long argmax_key(float v, int i) {
    uint32_t b = __float_as_uint(v);
    b = (b & 0x80000000u) ? ~b : (b | 0x80000000u);
    return ((unsigned long long)b << 32) | (uint32_t)(0x7fffffff - i);
}
__device__ __forceinline__ unsigned long long wave_max_u64(unsigned long long k) {
#pragma unroll
    for (int off = 32; off > 0; off >>= 1) {
        const unsigned long long o = __shfl_xor(k, off, 64);
        k = o > k ? o : k;
    }
    return k;
}
__global__ __launch_bounds__(256) void argmax_f32_partial_kernel(unsigned long long *__restrict__ keys, const float *__restrict__ logits,
                                                                  int vocab, int chunks) {
    __shared__ unsigned long long red[4];
    const int r = blockIdx.y, c = blockIdx.x;
    unsigned long long best = 0;
    for (int i = c * VMX_ARGMAX_CHUNK + threadIdx.x; i < min(vocab, (c + 1) * VMX_ARGMAX_CHUNK); i += 256) {
        const unsigned long long k = argmax_key(logits[(int64_t)r * vocab + i], i);
        best = k > best ? k : best;
    }
    best = wave_max_u64(best);
    if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = best;
    __syncthreads();
    if (threadIdx.x == 0) {
        for (int w2 = 1; w2 < 4; w2++) best = red[w2] > best ? red[w2] : best;
        keys[(int64_t)r * chunks + c] = best;
    }
}
__global__ __launch_bounds__(64) void argmax_f32_final_kernel(int32_t *__restrict__ out, const unsigned long long *__restrict__ keys, int chunks) {
    const int r = blockIdx.x;
    unsigned long long best = 0;
    for (int c = threadIdx.x; c < chunks; c += 64) best = keys[(int64_t)r * chunks + c] > best ? keys[(int64_t)r * chunks + c] : best;
    best = wave_max_u64(best);
    if (threadIdx.x == 0) out[r] = best ? 0x7fffffff - (int)(uint32_t)(best & 0xffffffffu) : 0;
}

__global__ __launch_bounds__(256) void zero_f32_kernel(float *__restrict__ p, int64_t n) {
    for (int64_t i = blockIdx.x * 256 + threadIdx.x; i < n; i += (int64_t)gridDim.x * 256) p[i] = 0.f;
}

// x[t] = embed[token] * scale (bf16 table, f32 rows); ids outside the table are clamped
__global__ __launch_bounds__(256) void embed_scaled_f32_kernel(float *__restrict__ x, const uint16_t *__restrict__ embed,
                                                                const int32_t *__restrict__ tokens, int width, int vocab, float scale) {
    const int t = blockIdx.x;
    int id = tokens[t];
    id = id < 0 ? 0 : (id >= vocab ? vocab - 1 : id);
    for (int i = threadIdx.x; i < width; i += 256) x[(int64_t)t * width + i] = vmx_bf16_to_f32(embed[(int64_t)id * width + i]) * scale;
}

// act[r, j] = f(gu[r, j]) * gu[r, ff + j]: the gated activation between the two products of a feed-forward whose gate and up
// projections were computed as one product; f = silu or the tanh form of gelu.  CLAMPED: g = min(gate, limit), u clamped to
// [-limit, limit], act = g sigmoid(slope g) (u + 1)
enum GluKind { GLU_SILU, GLU_GELU, GLU_CLAMPED };
template <GluKind KIND>
__global__ __launch_bounds__(256) void glu_kernel(void *__restrict__ act, int act_f32, const float *__restrict__ gu, int ff, float slope, float limit) {
    const int64_t r = blockIdx.x;             // rows on x: a prompt's (token, expert) pairs can pass the 65535 of the other axes
    const int j = blockIdx.y * 256 + threadIdx.x;
    if (j >= ff) return;
    float g = gu[r * 2 * ff + j], u = gu[r * 2 * ff + ff + j], f;
    if constexpr (KIND == GLU_GELU) f = 0.5f * g * (1.0f + tanhf(0.7978845608028654f * (g + 0.044715f * g * g * g)));
    else if constexpr (KIND == GLU_SILU) f = g / (1.0f + expf(-g));
    else {
        g = fminf(g, limit);
        f = g / (1.0f + expf(-slope * g));
        u = fminf(fmaxf(u, -limit), limit) + 1.0f;
    }
    const float v = f * u;
    if (act_f32) ((float *)act)[r * ff + j] = v;
    else ((uint16_t *)act)[r * ff + j] = vmx_f32_to_bf16(v);
}

// out[t] = [a[t] | b[t]] (two f32 rows of `width` numbers side by side), in f32 or bf16: the input of a product over both
__global__ __launch_bounds__(256) void concat2_rows_kernel(void *__restrict__ out, int out_f32, const float *__restrict__ a,
                                                            const float *__restrict__ b, int width) {
    const int t = blockIdx.x, i = blockIdx.y * 256 + threadIdx.x;
    if (i >= 2 * width) return;
    const float v = i < width ? a[(int64_t)t * width + i] : b[(int64_t)t * width + i - width];
    const int64_t o = (int64_t)t * 2 * width + i;
    if (out_f32) ((float *)out)[o] = v;
    else ((uint16_t *)out)[o] = vmx_f32_to_bf16(v);
}

// x <- cap * tanh(x * scale / cap) (cap 0: x * scale)
__global__ __launch_bounds__(256) void scale_softcap_kernel(float *__restrict__ x, int64_t n, float scale, float cap) {
    const int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x;
    if (i >= n) return;
    const float v = x[i] * scale;
    x[i] = cap > 0.f ? cap * tanhf(v / cap) : v;
}

}  // namespace

extern "C" int vmx_rotation_steps(const vmx_rotation *rot, float *steps, float *mul) {
    VMX_REQUIRE(rot && steps && mul, "rotation_steps: null pointer");
    const vmx_rotation &r = *rot;
    VMX_REQUIRE(r.dims >= 2 && r.dims % 2 == 0 && r.base > 1.0, "rotation_steps: %d rotated coordinates, base %g", r.dims, r.base);
    const int half = r.dims / 2;
    *mul = 1.f;
    double lo = 0, hi = 0;
    if (r.factor > 0.0) {
        VMX_REQUIRE(r.original > 0.0 && r.fast > 0.0 && r.slow > 0.0, "rotation_steps: bad stretch constants");
        auto idx = [&](double turns) { return r.dims * log(r.original / (2.0 * M_PI * turns)) / (2.0 * log(r.base)); };
        lo = std::max(floor(idx(r.fast)), 0.0);
        hi = std::min(ceil(idx(r.slow)), (double)(r.dims - 1));
        *mul = (float)(0.1 * log(r.factor) + 1.0);
    }
    for (int i = 0; i < half; i++) {
        double f = pow(r.base, -2.0 * i / r.dims);
        if (r.factor > 0.0) {
            const double ramp = std::min(std::max((i - lo) / std::max(hi - lo, 0.001), 0.0), 1.0);
            f = f / r.factor * ramp + f * (1.0 - ramp);
        }
        steps[i] = (float)f;
    }
    return VMX_OK;
}

int vmx_embed_scaled_f32(float *x, const uint16_t *embed, const int32_t *tokens, int T, int width, int vocab, float scale, hipStream_t st) {
    hipLaunchKernelGGL(embed_scaled_f32_kernel, dim3(T), dim3(256), 0, st, x, embed, tokens, width, vocab, scale);
    VMX_CHECK_LAUNCH("embed");
    return VMX_OK;
}

int vmx_glu_silu_rows(void *act, int act_f32, const float *gu, int rows, int ff, hipStream_t st) {
    if (rows <= 0) return VMX_OK;
    hipLaunchKernelGGL(glu_kernel<GLU_SILU>, dim3(rows, (ff + 255) / 256), dim3(256), 0, st, act, act_f32, gu, ff, 0.f, 0.f);
    VMX_CHECK_LAUNCH("glu silu");
    return VMX_OK;
}

int vmx_glu_gelu_rows(void *act, int act_f32, const float *gu, int rows, int ff, hipStream_t st) {
    if (rows <= 0) return VMX_OK;
    hipLaunchKernelGGL(glu_kernel<GLU_GELU>, dim3(rows, (ff + 255) / 256), dim3(256), 0, st, act, act_f32, gu, ff, 0.f, 0.f);
    VMX_CHECK_LAUNCH("glu gelu");
    return VMX_OK;
}

int vmx_glu_clamped_rows(void *act, int act_f32, const float *gu, int rows, int ff, float slope, float limit, hipStream_t st) {
    if (rows <= 0) return VMX_OK;
    hipLaunchKernelGGL(glu_kernel<GLU_CLAMPED>, dim3(rows, (ff + 255) / 256), dim3(256), 0, st, act, act_f32, gu, ff, slope, limit);
    VMX_CHECK_LAUNCH("glu clamped");
    return VMX_OK;
}

int vmx_rms_norm_f32in(void *out, int out_f32, const float *x, const int32_t *rows, const uint16_t *w, int w_scalar, int width, float eps,
                       int n, hipStream_t st) {
    if (n <= 0) return VMX_OK;
    hipLaunchKernelGGL(row_norm_f32in_kernel<false>, dim3(n), dim3(256), 0, st, out, out_f32, x, rows, w, w_scalar, width, eps);
    VMX_CHECK_LAUNCH("rms norm");
    return VMX_OK;
}

int vmx_layer_norm_f32in(void *out, int out_f32, const float *x, const int32_t *rows, const uint16_t *w, int width, float eps, int n, hipStream_t st) {
    if (n <= 0) return VMX_OK;
    hipLaunchKernelGGL(row_norm_f32in_kernel<true>, dim3(n), dim3(256), 0, st, out, out_f32, x, rows, w, 0, width, eps);
    VMX_CHECK_LAUNCH("layer norm");
    return VMX_OK;
}

int vmx_sandwich_norm(const VmxSandwich &a, int n, hipStream_t st) {
    VMX_REQUIRE(a.x && a.width >= 1 && (a.embed ? a.tokens && a.vocab >= 1 : a.y != nullptr), "sandwich norm: null pointer");
    VMX_REQUIRE((!a.w_next && !a.copy_h) || a.h, "sandwich norm: the next norm (or the copy) needs its output rows");
    VMX_REQUIRE(!a.side || (a.w_y && a.w_side && !a.embed && !a.pair_rows), "sandwich norm: two branches need their gains and plain rows");
    VMX_REQUIRE(!a.pair_rows || (a.pair_w && a.top >= 1), "sandwich norm: expert results need their weights");
    if (n <= 0) return VMX_OK;
    const bool vec = a.width % 4 == 0;   // every row then starts on a 16-byte (f32) / 8-byte (bf16) boundary
#define SW(held, v)                                                                                          \
    do {                                                                                                     \
        if (a.side) hipLaunchKernelGGL((sandwich_norm_kernel<held, v, true>), dim3(n), dim3(256), 0, st, a); \
        else hipLaunchKernelGGL((sandwich_norm_kernel<held, v, false>), dim3(n), dim3(256), 0, st, a);       \
    } while (0)
    if (vec && a.width <= 1024) SW(1, 4);
    else if (vec && a.width <= 2048) SW(2, 4);
    else if (vec && a.width <= 4096) SW(4, 4);
    else if (!vec && a.width <= 1024) SW(4, 1);
    else if (!vec && a.width <= 4096) SW(16, 1);
    else SW(0, 1);
#undef SW
    VMX_CHECK_LAUNCH("sandwich norm");
    return VMX_OK;
}

int vmx_group_norm_post(float *acc, float *x, void *h, int h_f32, const uint16_t *w, int groups, int width, float eps, float alpha, int n,
                        hipStream_t st) {
    VMX_REQUIRE(acc && x && h && groups >= 1 && width % groups == 0, "group norm: %d groups do not divide a row of %d", groups, width);
    if (n <= 0) return VMX_OK;
    hipLaunchKernelGGL(group_norm_post_kernel, dim3(n), dim3(256), 0, st, acc, x, h, h_f32, w, groups, width, eps, alpha);
    VMX_CHECK_LAUNCH("group norm");
    return VMX_OK;
}

int vmx_group_norm_rows(void *out, int out_f32, const float *x, const int32_t *rows, const uint16_t *w, int groups, int width, float eps, int n,
                        hipStream_t st) {
    VMX_REQUIRE(out && x && w && groups >= 1 && width % groups == 0, "group norm: %d groups do not divide a row of %d", groups, width);
    if (n <= 0) return VMX_OK;
    hipLaunchKernelGGL(group_norm_rows_kernel, dim3(n), dim3(256), 0, st, out, out_f32, x, rows, w, groups, width, eps);
    VMX_CHECK_LAUNCH("group norm rows");
    return VMX_OK;
}

int vmx_glu_silu_rows_scaled(void *act, int act_f32, const float *gu, int64_t ldgu, int up_off, int rows, int ff, const float *in_w,
                             const int32_t *in_ids, int in_limit, const float *out_gate, int64_t ldgate, hipStream_t st) {
    if (rows <= 0) return VMX_OK;
    hipLaunchKernelGGL(glu_silu_scaled_kernel, dim3(rows, (ff + 255) / 256), dim3(256), 0, st, act, act_f32, gu, ldgu, up_off, ff, in_w, in_ids,
                       in_limit, out_gate, ldgate);
    VMX_CHECK_LAUNCH("glu silu (scaled)");
    return VMX_OK;
}

int vmx_zero_f32(float *p, int64_t n, hipStream_t st) {
    hipLaunchKernelGGL(zero_f32_kernel, dim3(1024), dim3(256), 0, st, p, n);
    VMX_CHECK_LAUNCH("zero");
    return VMX_OK;
}

int vmx_moe_inverse(int32_t *inv, const int32_t *sorted, const int32_t *total, int numel, int cap, hipStream_t st) {
    hipLaunchKernelGGL(moe_inverse_kernel, dim3((cap + 255) / 256), dim3(256), 0, st, inv, sorted, total, numel);
    VMX_CHECK_LAUNCH("moe inverse");
    return VMX_OK;
}

int vmx_moe_combine_f32(float *x, const float *y, const int32_t *inv, const float *w, int k, const float *shared, const float *gate,
                        int64_t ldgate, int T, int width, hipStream_t st) {
    hipLaunchKernelGGL(moe_combine_f32_kernel, dim3(T, (width + 255) / 256), dim3(256), 0, st, x, y, inv, w, k, shared, gate, ldgate, width);
    VMX_CHECK_LAUNCH("moe combine");
    return VMX_OK;
}

int vmx_argmax_f32_rows(int32_t *out, unsigned long long *keys, const float *logits, int rows, int vocab, hipStream_t st) {
    const int chunks = (vocab + VMX_ARGMAX_CHUNK - 1) / VMX_ARGMAX_CHUNK;
    hipLaunchKernelGGL(argmax_f32_partial_kernel, dim3(chunks, rows), dim3(256), 0, st, keys, logits, vocab, chunks);
    hipLaunchKernelGGL(argmax_f32_final_kernel, dim3(rows), dim3(64), 0, st, out, keys, chunks);
    VMX_CHECK_LAUNCH("argmax");
    return VMX_OK;
}

int vmx_concat2_rows(void *out, int out_f32, const float *a, const float *b, int T, int width, hipStream_t st) {
    if (T <= 0) return VMX_OK;
    hipLaunchKernelGGL(concat2_rows_kernel, dim3(T, (2 * width + 255) / 256), dim3(256), 0, st, out, out_f32, a, b, width);
    VMX_CHECK_LAUNCH("concat rows");
    return VMX_OK;
}

int vmx_scale_softcap_f32(float *x, int64_t n, float scale, float cap, hipStream_t st) {
    if (n <= 0) return VMX_OK;
    hipLaunchKernelGGL(scale_softcap_kernel, dim3((unsigned)((n + 255) / 256)), dim3(256), 0, st, x, n, scale, cap);
    VMX_CHECK_LAUNCH("scale + soft cap");
    return VMX_OK;
}
