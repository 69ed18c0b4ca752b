// A sublayer's result on its way into the residual stream.  The result is a sum of up to three kinds of pieces:
//
//   u[t] = sum_k choices[t * top + k]  +  id_wts[t] * x[t]  +  y[t]
//
// choices: float32 rows of a mixture of experts, one per (token, choice), added in their order; a choice whose id is
// negative has no row and is left out (ids null: every choice counts).  id_wts, x: a weight per token on the sublayer's
// own input (the choices that hand the input through).  y: a result that every token has (a shared expert's, or a
// mixer's).  Every kind is optional.
//
//   vt_sublayer_sum:     out[t] = u[t]
//   vt_output_norm_add:  h[t] <- h[t] + mult * (gain * u[t]) / sqrt(mean(u[t]^2) + eps), and copy[t] = h[t] in the copy's
//                        type: a norm on the sublayer's output, its addition to the float32 stream and the copy that the
//                        next sublayer's matrix products read, in one pass over the row.
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
    const float* gain;      // [W]
    void* copy;             // [n][W] or null
    int W, top, x_f32, y_f32, copy_f32;
    float mult, eps;
};

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

// element j of the row's sum
__device__ __forceinline__ float on_sum(const OutNormArgs& a, size_t t, int j) {
    float u = 0.f;
    if (a.choices)
        for (int k = 0; k < a.top; ++k) {
            const size_t p = t * a.top + k;
            if (!a.ids || a.ids[p] >= 0) u += a.choices[p * a.W + j];
        }
    if (a.id_wts) u = fmaf(a.id_wts[t], on_any(a.x, a.x_f32, t * a.W + j), u);
    if (a.y) u += on_any(a.y, a.y_f32, t * a.W + j);
    return u;
}

// NORM: the norm and the addition to h; otherwise the sum alone.  Any width; the sum is formed twice.
template <bool NORM>
__global__ __launch_bounds__(256) void output_norm_kernel(OutNormArgs a) {
    __shared__ float red[16];
    const size_t t = blockIdx.x;
    if constexpr (!NORM) {
        for (int j = threadIdx.x; j < a.W; j += 256) a.h[t * a.W + j] = on_sum(a, t, j);
        return;
    }
    float ss = 0.f;
    for (int j = threadIdx.x; j < a.W; j += 256) {
        const float u = on_sum(a, t, j);
        ss = fmaf(u, u, ss);
    }
    ss = block_sum(ss, red);
    const float r = a.mult / sqrtf(ss / (float)a.W + a.eps);
    for (int j = threadIdx.x; j < a.W; j += 256) {
        const float v = fmaf(a.gain[j] * on_sum(a, t, j), r, a.h[t * a.W + j]);
        a.h[t * a.W + j] = v;
        if (a.copy) {
            if (a.copy_f32) ((float*)a.copy)[t * a.W + j] = v;
            else ((bf16_t*)a.copy)[t * a.W + j] = f32_to_bf16(v);
        }
    }
}

// Widths that are multiples of 4 up to 1024 NV: a thread keeps NV pieces of four elements in registers between the sum
// of squares and the scaling, and everything that does not depend on it (stream, gains) is asked for in front of it.
template <bool NORM, int NV>
__global__ __launch_bounds__(256) void output_norm_vec_kernel(OutNormArgs a) {
    __shared__ float red[16];
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
        if (a.y) {
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
        if (a.copy) {
            if (a.copy_f32) {
                *(float4*)((float*)a.copy + row + 4 * q) = v;
            } else {
                uint2 o;
                o.x = vt_pack2(v.x, v.y);
                o.y = vt_pack2(v.z, v.w);
                *(uint2*)((bf16_t*)a.copy + row + 4 * q) = o;
            }
        }
    }
}

template <bool NORM>
static void out_norm_launch(const OutNormArgs& a, int n, hipStream_t stream) {
    const bool vec = a.W % 4 == 0 && a.W <= 8192 &&
                     !(((uintptr_t)a.h | (uintptr_t)a.choices | (uintptr_t)a.x | (uintptr_t)a.y | (uintptr_t)a.gain | (uintptr_t)a.copy) & 15);
    if (vec && a.W <= 1024) output_norm_vec_kernel<NORM, 1><<<n, 256, 0, stream>>>(a);
    else if (vec && a.W <= 2048) output_norm_vec_kernel<NORM, 2><<<n, 256, 0, stream>>>(a);
    else if (vec && a.W <= 4096) output_norm_vec_kernel<NORM, 4><<<n, 256, 0, stream>>>(a);
    else if (vec) output_norm_vec_kernel<NORM, 8><<<n, 256, 0, stream>>>(a);
    else output_norm_kernel<NORM><<<n, 256, 0, stream>>>(a);
}

static int out_norm_args(OutNormArgs& a, const char* who, float* h, const float* choices, const int* ids, int top, const float* id_wts,
                         const void* x, int x_dtype, const void* y, int y_dtype, int n, int W) {
    VT_REQUIRE(n >= 0 && W > 0 && h, "%s: bad sizes n=%d W=%d", who, n, W);
    VT_REQUIRE(choices || id_wts || y, "%s: no pieces", who);
    VT_REQUIRE(!choices || top > 0, "%s: %d choices per token", who, top);
    VT_REQUIRE(!id_wts || (x && (x_dtype == VT_F32 || x_dtype == VT_BF16)), "%s: weights without an input of a known type", who);
    VT_REQUIRE(!y || y_dtype == VT_F32 || y_dtype == VT_BF16, "%s: unknown dtype %d", who, y_dtype);
    a.h = h; a.choices = choices; a.ids = ids; a.id_wts = id_wts; a.x = id_wts ? x : nullptr; a.y = y; a.gain = nullptr; a.copy = nullptr;
    a.W = W; a.top = top; a.x_f32 = x_dtype == VT_F32; a.y_f32 = y_dtype == VT_F32; a.copy_f32 = 0; a.mult = 1.f; a.eps = 0.f;
    return 0;
}

extern "C" int vt_sublayer_sum(float* out, const float* choices, const int* ids, int top, const float* id_wts, const void* x,
                               int x_dtype, const void* y, int y_dtype, int n, int W, hipStream_t stream) {
    OutNormArgs a;
    if (out_norm_args(a, "vt_sublayer_sum", out, choices, ids, top, id_wts, x, x_dtype, y, y_dtype, n, W)) return -1;
    if (n == 0) return 0;
    out_norm_launch<false>(a, n, stream);
    VT_CHECK_LAUNCH("vt_sublayer_sum");
    return 0;
}

extern "C" int vt_output_norm_add(float* h, const float* choices, const int* ids, int top, const float* id_wts, const void* x,
                                  int x_dtype, const void* y, int y_dtype, const float* gain, void* copy, int copy_dtype, int n,
                                  int W, float mult, float eps, hipStream_t stream) {
    OutNormArgs a;
    if (out_norm_args(a, "vt_output_norm_add", h, choices, ids, top, id_wts, x, x_dtype, y, y_dtype, n, W)) return -1;
    VT_REQUIRE(gain, "vt_output_norm_add: no gains");
    VT_REQUIRE(!copy || copy_dtype == VT_F32 || copy_dtype == VT_BF16, "vt_output_norm_add: unknown copy dtype %d", copy_dtype);
    if (n == 0) return 0;
    a.gain = gain; a.copy = copy; a.copy_f32 = copy_dtype == VT_F32; a.mult = mult; a.eps = eps;
    out_norm_launch<true>(a, n, stream);
    VT_CHECK_LAUNCH("vt_output_norm_add");
    return 0;
}
