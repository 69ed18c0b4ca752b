// Linear attention with a constant decay per head as a token mixer with per-request state, for prompts and decoding.
//
// Per head, a matrix state S [D][Dv] in float32 is carried from token to token:
//     S <- g S + k v^T;   o = S^T q          (the read-out sees the token's own write)
// with q, k and v the activations (SiLU, or none) of a projection's columns and g a constant of the model.
//
//   vt_decayed_attn:  steps that bring single tokens, one per request (decoding): a row of 16 lanes per state column, each
//                     lane with a sixteenth of its elements; every load is asked for at once.  Otherwise the same
//                     arrangement token by token, in tiles of 16 through LDS.
//
// The state of a head is kept [Dv][D]: a column's D elements lie together.
#include "vt_common.h"
#include <math.h>

VT_DEFINE_LAST_ERROR()

#define ROWS 16             // rows of 16 lanes in a block: state columns

__device__ __forceinline__ float silu_f(float z) { return z / (1.0f + expf(-z)); }

// the sum of v over the 16 lanes of a row (lanes 16 r .. 16 r + 15), in every one of them: four rotations within the row
__device__ __forceinline__ float row16_sum(float v) {
    v += __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, v), 0x128, 0xf, 0xf, false));
    v += __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, v), 0x124, 0xf, 0xf, false));
    v += __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, v), 0x122, 0xf, 0xf, false));
    v += __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, v), 0x121, 0xf, 0xf, false));
    return v;
}

// Which state element lane r of a row holds as its i-th: groups of four consecutive elements dealt out to the lanes in
// turn, so that a row reads 256 consecutive bytes at a time; heads of up to 64 elements: DS consecutive ones.
template <int DS>
__device__ __forceinline__ constexpr int lane_elem(int r, int i) {
    return DS <= 4 ? DS * r + i : 4 * (r + 16 * (i / 4)) + (i % 4);
}

struct DecayedArgs {
    const void* x;          // [n][ldx]: H heads of D queries from q_col, of D keys from k_col, of Dv values from v_col
    const float* decay;     // [H]
    float* state;           // slot s: state + s * slot_stride, [H][Dv][D]
    const int* entry_start;
    const int* slots;
    float* o;               // [n][H][Dv]
    long long ldx, slot_stride;
    int q_col, k_col, v_col;
    int H, D, Dv, silu;
};

// One token per entry: entry e's is token e.
template <typename TI, int DS>
__global__ __launch_bounds__(256) void decayed_step_kernel(DecayedArgs a) {
    const int e = blockIdx.x, h = blockIdx.y;
    const int tid = threadIdx.x, r = tid & 15;
    const int col = blockIdx.z * ROWS + (tid >> 4);
    const int D = a.D, Dv = a.Dv;
    const TI* x = (const TI*)a.x + (size_t)e * a.ldx;
    float* S = a.state + (size_t)a.slots[e] * a.slot_stride + ((size_t)h * Dv + col) * D;
    if (col >= Dv) return;      // (a row of lanes leaves together)
    float s[DS], k[DS], q[DS];
#pragma unroll
    for (int i = 0; i < DS; ++i) {
        const int d = lane_elem<DS>(r, i);
        const bool in = d < D;
        s[i] = in ? S[d] : 0.f;
        k[i] = in ? load_f32<TI>(x, a.k_col + (size_t)h * D + d) : 0.f;
        q[i] = in ? load_f32<TI>(x, a.q_col + (size_t)h * D + d) : 0.f;
    }
    float v = load_f32<TI>(x, a.v_col + (size_t)h * Dv + col);
    const float g = a.decay[h];
    if (a.silu) v = silu_f(v);
    float acc = 0.f;
#pragma unroll
    for (int i = 0; i < DS; ++i) {
        if (a.silu) {
            k[i] = silu_f(k[i]);
            q[i] = silu_f(q[i]);
        }
        s[i] = fmaf(g, s[i], k[i] * v);
        acc = fmaf(q[i], s[i], acc);
        const int d = lane_elem<DS>(r, i);
        if (d < D) S[d] = s[i];
    }
    acc = row16_sum(acc);
    if (r == 0) a.o[((size_t)e * a.H + h) * Dv + col] = acc;
}

// Any portions: token by token, the same instructions in the same order whatever the tile, so nothing depends on how a
// request was cut.  A tile's inputs (16 tokens x 16 lanes bring them) are asked for while the tile in front is worked through.
template <typename TI, int DS>
__global__ __launch_bounds__(256) void decayed_scan_kernel(DecayedArgs a) {
    constexpr int DP = 16 * DS, TILE = 16;
    __shared__ __attribute__((aligned(16))) float qs[TILE][DP];
    __shared__ __attribute__((aligned(16))) float ks[TILE][DP];
    __shared__ float vs[TILE][ROWS];

    const int e = blockIdx.x, h = blockIdx.y, col0 = blockIdx.z * ROWS;
    const int tid = threadIdx.x, r = tid & 15, cl = tid >> 4;
    const int D = a.D, Dv = a.Dv, H = a.H;
    const int start = a.entry_start[e], end = a.entry_start[e + 1];
    float* S_head = a.state + (size_t)a.slots[e] * a.slot_stride + (size_t)h * Dv * D;
    const TI* x = (const TI*)a.x;
    const int col = col0 + cl;
    const float g = a.decay[h];
    const bool act = a.silu != 0;

    float S[DS];
#pragma unroll
    for (int i = 0; i < DS; ++i) {
        const int d = lane_elem<DS>(r, i);
        S[i] = (col < Dv && d < D) ? S_head[(size_t)col * D + d] : 0.f;
    }
    float in_q[DS], in_k[DS], in_v = 0.f;
    auto fetch = [&](int t0) {
        const int t = t0 + cl;
        const bool ok = t < end;
        const size_t row = (size_t)(ok ? t : start) * a.ldx;
#pragma unroll
        for (int i = 0; i < DS; ++i) {
            const int d = lane_elem<DS>(r, i);
            const bool in = ok && d < D;
            in_q[i] = in ? load_f32<TI>(x, row + a.q_col + (size_t)h * D + d) : 0.f;
            in_k[i] = in ? load_f32<TI>(x, row + a.k_col + (size_t)h * D + d) : 0.f;
        }
        const int j = col0 + r;
        in_v = (ok && j < Dv) ? load_f32<TI>(x, row + a.v_col + (size_t)h * Dv + j) : 0.f;
    };
    fetch(start);
    for (int t0 = start; t0 < end; t0 += TILE) {
        const int nt = min(TILE, end - t0);
        __syncthreads();        // the tile before has been read
#pragma unroll
        for (int i = 0; i < DS; ++i) {
            const int d = lane_elem<DS>(r, i);
            qs[cl][d] = act ? silu_f(in_q[i]) : in_q[i];
            ks[cl][d] = act ? silu_f(in_k[i]) : in_k[i];
        }
        vs[cl][r] = act ? silu_f(in_v) : in_v;
        __syncthreads();
        if (t0 + TILE < end) fetch(t0 + TILE);
        auto token = [&](int tt) {
            const float v = vs[tt][cl];
            float acc = 0.f;
#pragma unroll
            for (int i = 0; i < DS; ++i) {
                const int d = lane_elem<DS>(r, i);
                S[i] = fmaf(g, S[i], ks[tt][d] * v);
                acc = fmaf(qs[tt][d], S[i], acc);
            }
            acc = row16_sum(acc);
            if (r == 0 && col < Dv) a.o[((size_t)(t0 + tt) * H + h) * Dv + col] = acc;
        };
        if (nt == TILE) {
#pragma unroll
            for (int tt = 0; tt < TILE; ++tt) token(tt);
        } else {
            for (int tt = 0; tt < nt; ++tt) token(tt);
        }
    }
#pragma unroll
    for (int i = 0; i < DS; ++i) {
        const int d = lane_elem<DS>(r, i);
        if (col < Dv && d < D) S_head[(size_t)col * D + d] = S[i];
    }
}

// single: every entry brings one token (entry e's is token e)
extern "C" int vt_decayed_attn(const void* x, int dtype, long long ldx, int q_col, int k_col, int v_col, const float* decay,
                               float* state, long long slot_stride, const int* entry_start, const int* slots, float* o,
                               int n_entries, int H, int D, int Dv, int silu, int single, hipStream_t stream) {
    VT_REQUIRE(n_entries >= 0 && H > 0 && H <= 65535, "vt_decayed_attn: bad heads %d", H);
    VT_REQUIRE(D > 0 && D <= 256 && Dv > 0 && Dv <= 65535 * ROWS, "vt_decayed_attn: head sizes %d/%d (keys up to 256)", D, Dv);
    VT_REQUIRE(slot_stride >= (long long)H * D * Dv, "vt_decayed_attn: state slots are too short");
    VT_REQUIRE(min(q_col, min(k_col, v_col)) >= 0 && ldx >= max(q_col, k_col) + (long long)H * D && ldx >= v_col + (long long)H * Dv,
               "vt_decayed_attn: rows are too short for their columns");
    if (n_entries == 0) return 0;
    DecayedArgs a;
    a.x = x; a.decay = decay; a.state = state; a.entry_start = entry_start; a.slots = slots; a.o = o; a.ldx = ldx;
    a.slot_stride = slot_stride; a.q_col = q_col; a.k_col = k_col; a.v_col = v_col; a.H = H; a.D = D; a.Dv = Dv; a.silu = silu;
    const int share = (D + 15) / 16;
    const dim3 grid(n_entries, H, (Dv + ROWS - 1) / ROWS);
#define VT_DECAYED_DS(KERNEL, TI)                                                            \
    do {                                                                                     \
        if (share <= 1) KERNEL<TI, 1><<<grid, 256, 0, stream>>>(a);                          \
        else if (share <= 2) KERNEL<TI, 2><<<grid, 256, 0, stream>>>(a);                     \
        else if (share <= 4) KERNEL<TI, 4><<<grid, 256, 0, stream>>>(a);                     \
        else if (share <= 8) KERNEL<TI, 8><<<grid, 256, 0, stream>>>(a);                     \
        else KERNEL<TI, 16><<<grid, 256, 0, stream>>>(a);                                    \
    } while (0)
    if (dtype != VT_F32 && dtype != VT_BF16) return vt_fail("vt_decayed_attn: unknown dtype %d", dtype);
    if (single) {
        if (dtype == VT_F32) VT_DECAYED_DS(decayed_step_kernel, float);
        else VT_DECAYED_DS(decayed_step_kernel, bf16_t);
    } else {
        if (dtype == VT_F32) VT_DECAYED_DS(decayed_scan_kernel, float);
        else VT_DECAYED_DS(decayed_scan_kernel, bf16_t);
    }
#undef VT_DECAYED_DS
    VT_CHECK_LAUNCH("vt_decayed_attn");
    return 0;
}
