// A sublayer's result on its way into the residual stream.  The result is a sum of up to three kinds of pieces:
//
//   u[t] = sum_k choices[t * top + k]  +  id_wts[t] * x[t]  +  y[t]
//
// choices: float32 rows of a mixture of experts, one per (token, choice), added in their order; a choice whose id is
// negative has no row and is left out (ids null: every choice counts).  id_wts, x: a weight per token on the sublayer's
// own input (the choices that hand the input through).  y: a result that every token has (a shared expert's, or a
// mixer's).  Every kind is optional.  In y's place two results may stand, each normed first:
//   y[t] = y_scale * (y_gain * y1[t]) / sqrt(mean(y1[t]^2) + pair_eps) + y2_scale * (y2_gain * y2[t]) / sqrt(mean(y2[t]^2) + pair_eps)
//
//   vt_sublayer_sum:     out[t] = u[t]
//   vt_output_norm_add:  h[t] <- h[t] + mult * (gain * u[t]) / sqrt(mean(u[t]^2) + eps), and copy[t] = h[t] in the copy's
//                        type: a norm on the sublayer's output, its addition to the float32 stream and the copy that the
//                        next sublayer's matrix products read, in one pass over the row.  With next_gain the copy holds
//                        the norm in front of that sublayer instead: next_gain * h[t] / sqrt(mean(h[t]^2) + next_eps).
// x may be h itself: a thread reads the elements that it writes, and only those.
// A block per token; sums are taken in an order that depends on the width alone.
#include "vt_common.h"

VT_DEFINE_LAST_ERROR()

struct OutNormArgs {
    float* h;               // [n][W] (or the sum's destination)
    const float* choices;   // [n * top][W] or null
    const int* ids;         // [n * top] or null
    const float* id_wts;    // [n] or null
    const void* x;          // [n][W], read where id_wts is given
    const void* y;          // [n][W] or null
    const void* y2;         // [n][W] or null: y and y2 are a pair of results to be normed
    const float* y_gain;    // [W] each, with y2
    const float* y2_gain;
    const float* gain;      // [W]
    void* copy;             // [n][W] or null
    const float* next_gain; // [W] or null
    int W, top, x_f32, y_f32, y2_f32, copy_f32;
    float mult, eps, y_scale, y2_scale, pair_eps, next_eps;
};

// the sums of two values over the block, in block_sum's order; red: 32 floats
__device__ __forceinline__ float2 block_sum2(float a, float b, float* red) {
    a = wave_sum(a);
    b = wave_sum(b);
    const int w = threadIdx.x >> 6, nw = blockDim.x >> 6;
    __syncthreads();
    if ((threadIdx.x & 63) == 0) { red[w] = a; red[16 + w] = b; }
    __syncthreads();
    float2 t = make_float2(0.f, 0.f);
    for (int i = 0; i < nw; ++i) { t.x += red[i]; t.y += red[16 + i]; }
    return t;
}

__device__ __forceinline__ float4 on_load4(const float* p) { return *(const float4*)p; }
__device__ __forceinline__ float4 on_load4(const bf16_t* p) {
    const uint2 u = *(const uint2*)p;
    return make_float4(lowp_lo(u.x), lowp_hi(u.x), lowp_lo(u.y), lowp_hi(u.y));
}
__device__ __forceinline__ float4 on_any4(const void* p, int f32, size_t i) {
    return f32 ? on_load4((const float*)p + i) : on_load4((const bf16_t*)p + i);
}
__device__ __forceinline__ float on_any(const void* p, int f32, size_t i) {
    return f32 ? ((const float*)p)[i] : bf16_to_f32(((const bf16_t*)p)[i]);
}

// four elements of the copy, in its type
__device__ __forceinline__ void on_store4(const OutNormArgs& a, size_t i, float4 v) {
    if (a.copy_f32) {
        *(float4*)((float*)a.copy + i) = v;
    } else {
        uint2 o;
        o.x = vt_pack2(v.x, v.y);
        o.y = vt_pack2(v.z, v.w);
        *(uint2*)((bf16_t*)a.copy + i) = o;
    }
}

// element j of the row's sum; r1, r2: what a pair's elements are multiplied by beside their gains
__device__ __forceinline__ float on_sum(const OutNormArgs& a, size_t t, int j, float r1, float r2) {
    float u = 0.f;
    if (a.choices)
        for (int k = 0; k < a.top; ++k) {
            const size_t p = t * a.top + k;
            if (!a.ids || a.ids[p] >= 0) u += a.choices[p * a.W + j];
        }
    if (a.id_wts) u = fmaf(a.id_wts[t], on_any(a.x, a.x_f32, t * a.W + j), u);
    if (a.y2) u += a.y_gain[j] * on_any(a.y, a.y_f32, t * a.W + j) * r1 + a.y2_gain[j] * on_any(a.y2, a.y2_f32, t * a.W + j) * r2;
    else if (a.y) u += on_any(a.y, a.y_f32, t * a.W + j);
    return u;
}

// NORM: the norm and the addition to h; otherwise the sum alone.  Any width; the sum is formed twice.
template <bool NORM>
__global__ __launch_bounds__(256) void output_norm_kernel(OutNormArgs a) {
    __shared__ float red[32];
    const size_t t = blockIdx.x;
    float r1 = 0.f, r2 = 0.f;
    if (a.y2) {
        float s1 = 0.f, s2 = 0.f;
        for (int j = threadIdx.x; j < a.W; j += 256) {
            const float p = on_any(a.y, a.y_f32, t * a.W + j), q = on_any(a.y2, a.y2_f32, t * a.W + j);
            s1 = fmaf(p, p, s1);
            s2 = fmaf(q, q, s2);
        }
        const float2 s = block_sum2(s1, s2, red);
        r1 = a.y_scale / sqrtf(s.x / (float)a.W + a.pair_eps);
        r2 = a.y2_scale / sqrtf(s.y / (float)a.W + a.pair_eps);
    }
    if constexpr (!NORM) {
        for (int j = threadIdx.x; j < a.W; j += 256) a.h[t * a.W + j] = on_sum(a, t, j, r1, r2);
        return;
    }
    float ss = 0.f;
    for (int j = threadIdx.x; j < a.W; j += 256) {
        const float u = on_sum(a, t, j, r1, r2);
        ss = fmaf(u, u, ss);
    }
    ss = block_sum(ss, red);
    const float r = a.mult / sqrtf(ss / (float)a.W + a.eps);
    float sn = 0.f;
    for (int j = threadIdx.x; j < a.W; j += 256) {
        const float v = fmaf(a.gain[j] * on_sum(a, t, j, r1, r2), r, a.h[t * a.W + j]);
        a.h[t * a.W + j] = v;
        sn = fmaf(v, v, sn);
        if (a.copy && !a.next_gain) {
            if (a.copy_f32) ((float*)a.copy)[t * a.W + j] = v;
            else ((bf16_t*)a.copy)[t * a.W + j] = f32_to_bf16(v);
        }
    }
    if (a.copy && a.next_gain) {
        sn = block_sum(sn, red);
        const float rn = 1.0f / sqrtf(sn / (float)a.W + a.next_eps);
        for (int j = threadIdx.x; j < a.W; j += 256) {
            const float v = a.next_gain[j] * a.h[t * a.W + j] * rn;        // (this thread has written the element)
            if (a.copy_f32) ((float*)a.copy)[t * a.W + j] = v;
            else ((bf16_t*)a.copy)[t * a.W + j] = f32_to_bf16(v);
        }
    }
}

// Widths that are multiples of 4 up to 1024 NV: a thread keeps NV pieces of four elements in registers between the sum
// of squares and the scaling, and everything that does not depend on it (stream, gains) is asked for in front of it.
template <bool NORM, int NV>
__global__ __launch_bounds__(256) void output_norm_vec_kernel(OutNormArgs a) {
    __shared__ float red[32];
    const size_t t = blockIdx.x, row = t * a.W;
    const int W4 = a.W >> 2;
    float4 u[NV], hv[NV], gn[NV];
    const float iw = a.id_wts ? a.id_wts[t] : 0.f;
#pragma unroll
    for (int i = 0; i < NV; ++i) {
        const int q = threadIdx.x + 256 * i;
        u[i] = make_float4(0.f, 0.f, 0.f, 0.f);
        if (NORM && q < W4) {
            hv[i] = on_load4(a.h + row + 4 * q);
            gn[i] = on_load4(a.gain + 4 * q);
        }
    }
    if (a.choices) {
#pragma unroll 4
        for (int k = 0; k < a.top; ++k) {
            const size_t p = t * a.top + k;
            if (a.ids && a.ids[p] < 0) continue;
#pragma unroll
            for (int i = 0; i < NV; ++i) {
                const int q = threadIdx.x + 256 * i;
                if (q < W4) {
                    const float4 v = on_load4(a.choices + p * a.W + 4 * q);
                    u[i].x += v.x; u[i].y += v.y; u[i].z += v.z; u[i].w += v.w;
                }
            }
        }
    }
    if (a.y2) {
        // (the pair's gains are asked for with its elements, in front of the barriers)
        float4 p[NV], s[NV], gp[NV], gs[NV];
        float s1 = 0.f, s2 = 0.f;
#pragma unroll
        for (int i = 0; i < NV; ++i) {
            const int q = threadIdx.x + 256 * i;
            if (q >= W4) continue;
            p[i] = on_any4(a.y, a.y_f32, row + 4 * q);
            s[i] = on_any4(a.y2, a.y2_f32, row + 4 * q);
            gp[i] = on_load4(a.y_gain + 4 * q);
            gs[i] = on_load4(a.y2_gain + 4 * q);
            s1 = fmaf(p[i].x, p[i].x, fmaf(p[i].y, p[i].y, fmaf(p[i].z, p[i].z, fmaf(p[i].w, p[i].w, s1))));
            s2 = fmaf(s[i].x, s[i].x, fmaf(s[i].y, s[i].y, fmaf(s[i].z, s[i].z, fmaf(s[i].w, s[i].w, s2))));
        }
        const float2 sums = block_sum2(s1, s2, red);
        const float r1 = a.y_scale / sqrtf(sums.x / (float)a.W + a.pair_eps), r2 = a.y2_scale / sqrtf(sums.y / (float)a.W + a.pair_eps);
#pragma unroll
        for (int i = 0; i < NV; ++i) {
            const int q = threadIdx.x + 256 * i;
            if (q >= W4) continue;
            u[i].x += gp[i].x * p[i].x * r1 + gs[i].x * s[i].x * r2;
            u[i].y += gp[i].y * p[i].y * r1 + gs[i].y * s[i].y * r2;
            u[i].z += gp[i].z * p[i].z * r1 + gs[i].z * s[i].z * r2;
            u[i].w += gp[i].w * p[i].w * r1 + gs[i].w * s[i].w * r2;
        }
    }
    float ss = 0.f;
#pragma unroll
    for (int i = 0; i < NV; ++i) {
        const int q = threadIdx.x + 256 * i;
        if (q >= W4) continue;
        if (a.id_wts) {
            const float4 v = on_any4(a.x, a.x_f32, row + 4 * q);
            u[i].x = fmaf(iw, v.x, u[i].x); u[i].y = fmaf(iw, v.y, u[i].y);
            u[i].z = fmaf(iw, v.z, u[i].z); u[i].w = fmaf(iw, v.w, u[i].w);
        }
        if (a.y && !a.y2) {
            const float4 v = on_any4(a.y, a.y_f32, row + 4 * q);
            u[i].x += v.x; u[i].y += v.y; u[i].z += v.z; u[i].w += v.w;
        }
        if (!NORM) *(float4*)(a.h + row + 4 * q) = u[i];
        ss = fmaf(u[i].x, u[i].x, ss);
        ss = fmaf(u[i].y, u[i].y, ss);
        ss = fmaf(u[i].z, u[i].z, ss);
        ss = fmaf(u[i].w, u[i].w, ss);
    }
    if constexpr (!NORM) return;
    ss = block_sum(ss, red);
    const float r = a.mult / sqrtf(ss / (float)a.W + a.eps);
    const bool behind = a.copy && a.next_gain;
    float sn = 0.f;
#pragma unroll
    for (int i = 0; i < NV; ++i) {
        const int q = threadIdx.x + 256 * i;
        if (q >= W4) continue;
        float4 v;
        v.x = fmaf(gn[i].x * u[i].x, r, hv[i].x);
        v.y = fmaf(gn[i].y * u[i].y, r, hv[i].y);
        v.z = fmaf(gn[i].z * u[i].z, r, hv[i].z);
        v.w = fmaf(gn[i].w * u[i].w, r, hv[i].w);
        *(float4*)(a.h + row + 4 * q) = v;
        if (behind) {
            gn[i] = on_load4(a.next_gain + 4 * q);
            u[i] = v;
            sn = fmaf(v.x, v.x, fmaf(v.y, v.y, fmaf(v.z, v.z, fmaf(v.w, v.w, sn))));
        } else if (a.copy) {
            on_store4(a, row + 4 * q, v);
        }
    }
    if (!behind) return;
    sn = block_sum(sn, red);
    const float rn = 1.0f / sqrtf(sn / (float)a.W + a.next_eps);
#pragma unroll
    for (int i = 0; i < NV; ++i) {
        const int q = threadIdx.x + 256 * i;
        if (q >= W4) continue;
        on_store4(a, row + 4 * q, make_float4(gn[i].x * u[i].x * rn, gn[i].y * u[i].y * rn, gn[i].z * u[i].z * rn, gn[i].w * u[i].w * rn));
    }
}

template <bool NORM>
static void out_norm_launch(const OutNormArgs& a, int n, hipStream_t stream) {
    const bool vec = a.W % 4 == 0 && a.W <= 8192 &&
                     !(((uintptr_t)a.h | (uintptr_t)a.choices | (uintptr_t)a.x | (uintptr_t)a.y | (uintptr_t)a.gain | (uintptr_t)a.copy |
                        (uintptr_t)a.y2 | (uintptr_t)a.y_gain | (uintptr_t)a.y2_gain | (uintptr_t)a.next_gain) & 15);
    if (vec && a.W <= 1024) output_norm_vec_kernel<NORM, 1><<<n, 256, 0, stream>>>(a);
    else if (vec && a.W <= 2048) output_norm_vec_kernel<NORM, 2><<<n, 256, 0, stream>>>(a);
    else if (vec && a.W <= 4096) output_norm_vec_kernel<NORM, 4><<<n, 256, 0, stream>>>(a);
    else if (vec) output_norm_vec_kernel<NORM, 8><<<n, 256, 0, stream>>>(a);
    else output_norm_kernel<NORM><<<n, 256, 0, stream>>>(a);
}

static int out_norm_args(OutNormArgs& a, const char* who, float* h, const float* choices, const int* ids, int top, const float* id_wts,
                         const void* x, int x_dtype, const void* y, int y_dtype, const void* y2, int y2_dtype,
                         const float* y_gain, const float* y2_gain, float y_scale, float y2_scale, float pair_eps, int n, int W) {
    VT_REQUIRE(n >= 0 && W > 0 && h, "%s: bad sizes n=%d W=%d", who, n, W);
    VT_REQUIRE(choices || id_wts || y, "%s: no pieces", who);
    VT_REQUIRE(!choices || top > 0, "%s: %d choices per token", who, top);
    VT_REQUIRE(!id_wts || (x && (x_dtype == VT_F32 || x_dtype == VT_BF16)), "%s: weights without an input of a known type", who);
    VT_REQUIRE(!y || y_dtype == VT_F32 || y_dtype == VT_BF16, "%s: unknown dtype %d", who, y_dtype);
    VT_REQUIRE(!y2 || (y && y_gain && y2_gain && (y2_dtype == VT_F32 || y2_dtype == VT_BF16) && pair_eps >= 0.f),
               "%s: a pair of results without its gains or of an unknown type", who);
    a.y2 = y2; a.y_gain = y_gain; a.y2_gain = y2_gain; a.y2_f32 = y2_dtype == VT_F32; a.y_scale = y_scale; a.y2_scale = y2_scale;
    a.pair_eps = pair_eps; a.next_gain = nullptr; a.next_eps = 0.f;
    a.h = h; a.choices = choices; a.ids = ids; a.id_wts = id_wts; a.x = id_wts ? x : nullptr; a.y = y; a.gain = nullptr; a.copy = nullptr;
    a.W = W; a.top = top; a.x_f32 = x_dtype == VT_F32; a.y_f32 = y_dtype == VT_F32; a.copy_f32 = 0; a.mult = 1.f; a.eps = 0.f;
    return 0;
}

extern "C" int vt_sublayer_sum(float* out, const float* choices, const int* ids, int top, const float* id_wts, const void* x,
                               int x_dtype, const void* y, int y_dtype, const void* y2, int y2_dtype, const float* y_gain,
                               const float* y2_gain, float y_scale, float y2_scale, float pair_eps, int n, int W, hipStream_t stream) {
    OutNormArgs a;
    if (out_norm_args(a, "vt_sublayer_sum", out, choices, ids, top, id_wts, x, x_dtype, y, y_dtype, y2, y2_dtype, y_gain, y2_gain,
                      y_scale, y2_scale, pair_eps, n, W)) return -1;
    if (n == 0) return 0;
    out_norm_launch<false>(a, n, stream);
    VT_CHECK_LAUNCH("vt_sublayer_sum");
    return 0;
}

extern "C" int vt_output_norm_add(float* h, const float* choices, const int* ids, int top, const float* id_wts, const void* x,
                                  int x_dtype, const void* y, int y_dtype, const void* y2, int y2_dtype, const float* y_gain,
                                  const float* y2_gain, float y_scale, float y2_scale, float pair_eps, const float* gain, void* copy,
                                  int copy_dtype, const float* next_gain, float next_eps, int n, int W, float mult, float eps,
                                  hipStream_t stream) {
    OutNormArgs a;
    if (out_norm_args(a, "vt_output_norm_add", h, choices, ids, top, id_wts, x, x_dtype, y, y_dtype, y2, y2_dtype, y_gain, y2_gain,
                      y_scale, y2_scale, pair_eps, n, W)) return -1;
    VT_REQUIRE(!next_gain || copy, "vt_output_norm_add: a norm behind without a place for it");
    VT_REQUIRE(gain, "vt_output_norm_add: no gains");
    VT_REQUIRE(!copy || copy_dtype == VT_F32 || copy_dtype == VT_BF16, "vt_output_norm_add: unknown copy dtype %d", copy_dtype);
    if (n == 0) return 0;
    a.next_gain = next_gain; a.next_eps = next_eps; a.gain = gain; a.copy = copy; a.copy_f32 = copy_dtype == VT_F32; a.mult = mult; a.eps = eps;
    out_norm_launch<true>(a, n, stream);
    VT_CHECK_LAUNCH("vt_output_norm_add");
    return 0;
}
