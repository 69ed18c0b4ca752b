// Linear attention with a constant decay per head as a token mixer with per-request state, for prompts and decoding.
//
// Per head, a matrix state S [D][Dv] in float32 is carried from token to token:
//     S <- g S + k v^T;   o = S^T q          (the read-out sees the token's own write)
// with q, k and v the activations (SiLU, or none) of a projection's columns and g a constant of the model.
//
//   vt_decayed_attn:  steps that bring single tokens, one per request (decoding): a row of 16 lanes per state column, each
//                     lane with a sixteenth of its elements; every load is asked for at once.  Otherwise the same
//                     arrangement token by token, in tiles of 16 through LDS.
//   vt_decayed_attn_chunked:  portions of prompts on the matrix cores, in float32 (v_mfma_f32_16x16x4): a request's tokens are
//                     cut into chunks of 64, and with i, j counted inside a chunk of n tokens and S_0 the state in front of it
//                         o_i = g^(i+1) S_0^T q_i + sum_{j <= i} g^(i-j) (q_i . k_j) v_j
//                         S_n = g^n S_0 + sum_j g^(n-1-j) k_j v_j^T
//                     Three launches: every chunk's sum of k v^T; the states in front of the chunks, one after the other,
//                     element by element; every chunk's outputs.
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

__device__ __forceinline__ void read4(const float* p, float* v) {
    const float4 f = *(const float4*)p;
    v[0] = f.x; v[1] = f.y; v[2] = f.z; v[3] = f.w;
}
__device__ __forceinline__ void read4(const bf16_t* p, float* v) {
    const uint2 u = *(const uint2*)p;
    v[0] = lowp_lo(u.x); v[1] = lowp_hi(u.x); v[2] = lowp_lo(u.y); v[3] = lowp_hi(u.y);
}

// One token per entry: entry e's is token e.  VEC: keys of a multiple of 4 elements that lie at multiples of 4 (a lane's
// groups of four are then 16-byte accesses, whole or not at all).
template <typename TI, int DS, bool VEC>
__global__ __launch_bounds__(256) void decayed_step_kernel(DecayedArgs a) {
    const int e = blockIdx.x, h = blockIdx.y;
    const int tid = threadIdx.x, r = tid & 15;
    const int col = blockIdx.z * ROWS + (tid >> 4);
    const int D = a.D, Dv = a.Dv;
    const TI* x = (const TI*)a.x + (size_t)e * a.ldx;
    float* S = a.state + (size_t)a.slots[e] * a.slot_stride + ((size_t)h * Dv + col) * D;
    if (col >= Dv) return;      // (a row of lanes leaves together)
    float s[DS], k[DS], q[DS];
    if constexpr (VEC) {
#pragma unroll
        for (int i = 0; i < DS; i += 4) {
            const int d = lane_elem<DS>(r, i);
#pragma unroll
            for (int j = 0; j < 4; ++j) s[i + j] = k[i + j] = q[i + j] = 0.f;
            if (d < D) {
                read4(S + d, s + i);
                read4(x + a.k_col + (size_t)h * D + d, k + i);
                read4(x + a.q_col + (size_t)h * D + d, q + i);
            }
        }
    } else {
#pragma unroll
        for (int i = 0; i < DS; ++i) {
            const int d = lane_elem<DS>(r, i);
            const bool in = d < D;
            s[i] = in ? S[d] : 0.f;
            k[i] = in ? load_f32<TI>(x, a.k_col + (size_t)h * D + d) : 0.f;
            q[i] = in ? load_f32<TI>(x, a.q_col + (size_t)h * D + d) : 0.f;
        }
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
    }
    if constexpr (VEC) {
#pragma unroll
        for (int i = 0; i < DS; i += 4) {
            const int d = lane_elem<DS>(r, i);
            if (d < D) *(float4*)(S + d) = make_float4(s[i], s[i + 1], s[i + 2], s[i + 3]);
        }
    } else {
#pragma unroll
        for (int i = 0; i < DS; ++i) {
            const int d = lane_elem<DS>(r, i);
            if (d < D) S[d] = s[i];
        }
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
    const bool vec = D % 4 == 0 && !((slot_stride | ldx | q_col | k_col) & 3) && !(((uintptr_t)state | (uintptr_t)x) & 15);
#define VT_DECAYED_STEP(TI)                                                                  \
    do {                                                                                     \
        if (share <= 1) decayed_step_kernel<TI, 1, false><<<grid, 256, 0, stream>>>(a);      \
        else if (share <= 2) decayed_step_kernel<TI, 2, false><<<grid, 256, 0, stream>>>(a); \
        else if (share <= 4 && vec) decayed_step_kernel<TI, 4, true><<<grid, 256, 0, stream>>>(a);   \
        else if (share <= 4) decayed_step_kernel<TI, 4, false><<<grid, 256, 0, stream>>>(a);         \
        else if (share <= 8 && vec) decayed_step_kernel<TI, 8, true><<<grid, 256, 0, stream>>>(a);   \
        else if (share <= 8) decayed_step_kernel<TI, 8, false><<<grid, 256, 0, stream>>>(a);         \
        else if (vec) decayed_step_kernel<TI, 16, true><<<grid, 256, 0, stream>>>(a);        \
        else decayed_step_kernel<TI, 16, false><<<grid, 256, 0, stream>>>(a);                \
    } while (0)
#define VT_DECAYED_SCAN(TI)                                                                  \
    do {                                                                                     \
        if (share <= 1) decayed_scan_kernel<TI, 1><<<grid, 256, 0, stream>>>(a);             \
        else if (share <= 2) decayed_scan_kernel<TI, 2><<<grid, 256, 0, stream>>>(a);        \
        else if (share <= 4) decayed_scan_kernel<TI, 4><<<grid, 256, 0, stream>>>(a);        \
        else if (share <= 8) decayed_scan_kernel<TI, 8><<<grid, 256, 0, stream>>>(a);        \
        else decayed_scan_kernel<TI, 16><<<grid, 256, 0, stream>>>(a);                       \
    } while (0)
    if (dtype != VT_F32 && dtype != VT_BF16) return vt_fail("vt_decayed_attn: unknown dtype %d", dtype);
    if (single) {
        if (dtype == VT_F32) VT_DECAYED_STEP(float);
        else VT_DECAYED_STEP(bf16_t);
    } else {
        if (dtype == VT_F32) VT_DECAYED_SCAN(float);
        else VT_DECAYED_SCAN(bf16_t);
    }
#undef VT_DECAYED_STEP
#undef VT_DECAYED_SCAN
    VT_CHECK_LAUNCH("vt_decayed_attn");
    return 0;
}

// ---------------------------------------------------------------------------
// Chunks of up to 64 tokens.  The matrix instruction takes k in steps of 4, one per group of 16 lanes; which four indices
// those are is free as long as both operands agree, so step q of a run of 16 takes the indices 4 grp + q: a lane's operands
// of four steps are then 4 consecutive elements where the sum runs over the key size, and the scores of one product (a
// lane holds rows 4 grp + q of its column) are the operands of the next as they stand.  Rows in LDS are padded by 4
// floats, which keeps both kinds of reads (16 rows of 16 bytes; 4 rows of 16 floats, 4 apart) off each other's banks.
// ---------------------------------------------------------------------------
#define CHUNK 64
#define VBLOCK 128          // value columns of a block
#define VROW (VBLOCK + 4)

typedef __attribute__((ext_vector_type(4))) float f32x4;
#define MFMA_F32(a, b, c) __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0)

struct ChunkArgs {
    const void* x;
    const float* powers;    // [H][CHUNK + 1]: g^0 .. g^64
    const int* chunks;      // [n_chunks][2]: first row, rows
    const int* chunk_start; // [entries + 1]: an entry's chunks
    const int* slots;
    float* state;
    float* work;            // [n_chunks][H][Dv][D]: a chunk's sum of k v^T, then the state in front of it
    float* o;
    long long ldx, slot_stride;
    int q_col, k_col, v_col;
    int H, D, Dv, silu;
};

__device__ __forceinline__ f32x4 read4(const float* p) { return *(const f32x4*)p; }
__device__ __forceinline__ f32x4 read4(const bf16_t* p) {
    const uint2 u = *(const uint2*)p;
    return (f32x4){lowp_lo(u.x), lowp_hi(u.x), lowp_lo(u.y), lowp_hi(u.y)};
}
__device__ __forceinline__ f32x4 act4(f32x4 v, bool silu) {
    if (silu) {
#pragma unroll
        for (int i = 0; i < 4; ++i) v[i] = silu_f(v[i]);
    }
    return v;
}

// `rows` tokens' columns [col, col + width) into LDS rows of `ld` floats, activated; what lies beyond the rows or the
// width (up to `padded` columns) is zero.  width and col are multiples of 4.
template <typename TI>
__device__ __forceinline__ void stage_rows(float* lds, int ld, const TI* x, long long ldx, int col, int width, int padded, int rows, bool silu) {
    const int per = padded >> 2;
    for (int i = threadIdx.x; i < CHUNK * per; i += 256) {
        const int t = i / per, c = (i - t * per) * 4;
        f32x4 v = {0.f, 0.f, 0.f, 0.f};
        if (t < rows && c < width) v = act4(read4(x + (size_t)t * ldx + col + c), silu);
        *(f32x4*)(lds + t * ld + c) = v;
    }
}

// a chunk's sum of g^(n-1-j) k_j v_j^T, [Dv][D]: a wave takes two tiles of 16 value columns and all of the key size
template <typename TI, int DT>
__global__ __launch_bounds__(256) void decayed_chunk_sum_kernel(ChunkArgs a) {
    constexpr int KROW = 16 * DT + 4;
    extern __shared__ __attribute__((aligned(16))) float lds[];
    float* ks = lds;                        // [CHUNK][KROW]
    float* vs = lds + CHUNK * KROW;         // [CHUNK][VROW]
    const int c = blockIdx.x, h = blockIdx.y, dv0 = blockIdx.z * VBLOCK;
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, r = lane & 15, grp = lane >> 4;
    const int first = a.chunks[2 * c], rows = a.chunks[2 * c + 1];
    const int D = a.D, Dv = a.Dv, vw = min(VBLOCK, Dv - dv0), vt = (vw + 15) / 16;
    const TI* x = (const TI*)a.x + (size_t)first * a.ldx;
    const float* pw = a.powers + (size_t)h * (CHUNK + 1);
    stage_rows<TI>(ks, KROW, x, a.ldx, a.k_col + h * D, D, 16 * DT, rows, a.silu != 0);
    stage_rows<TI>(vs, VROW, x, a.ldx, a.v_col + h * Dv + dv0, vw, 16 * vt, rows, a.silu != 0);
    __syncthreads();
    const int t0 = 2 * wave;
    if (t0 >= vt) return;
    const bool two = t0 + 1 < vt;
    f32x4 acc[2][DT];
#pragma unroll
    for (int u = 0; u < 2; ++u)
#pragma unroll
        for (int d = 0; d < DT; ++d) acc[u][d] = (f32x4){0.f, 0.f, 0.f, 0.f};
    for (int tb = 0; tb < rows; tb += 16) {
#pragma unroll
        for (int q = 0; q < 4; ++q) {
            const int j = tb + 4 * grp + q;
            const float w = j < rows ? pw[rows - 1 - j] : 0.f;
            const float* vr = vs + j * VROW + 16 * t0 + r;
            const float a0 = vr[0] * w, a1 = two ? vr[16] * w : 0.f;
            const float* kr = ks + j * KROW + r;
#pragma unroll
            for (int d = 0; d < DT; ++d) {
                const float b = kr[16 * d];
                acc[0][d] = MFMA_F32(a0, b, acc[0][d]);
                acc[1][d] = MFMA_F32(a1, b, acc[1][d]);
            }
        }
    }
    // acc[u][d][i]: value column 16 (t0 + u) + 4 grp + i, key element 16 d + r
    float* out = a.work + ((size_t)c * a.H + h) * Dv * D;
#pragma unroll
    for (int u = 0; u < 2; ++u)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            const int dv = dv0 + 16 * (t0 + u) + 4 * grp + i;
            if (dv >= Dv || (u && !two)) continue;
#pragma unroll
            for (int d = 0; d < DT; ++d)
                if (16 * d + r < D) out[(size_t)dv * D + 16 * d + r] = acc[u][d][i];
        }
}

// element by element: the states in front of an entry's chunks in the place of the chunks' sums, and the state behind the last
__global__ __launch_bounds__(256) void decayed_chunk_state_kernel(ChunkArgs a) {
    const int e = blockIdx.y;
    const size_t per = (size_t)a.Dv * a.D, all = per * a.H;
    const size_t idx = (size_t)blockIdx.x * 256 + threadIdx.x;
    if (idx >= all) return;
    const float* pw = a.powers + (idx / per) * (CHUNK + 1);
    float* st = a.state + (size_t)a.slots[e] * a.slot_stride + idx;
    float S = *st;
    const int c1 = a.chunk_start[e + 1];
    for (int c = a.chunk_start[e]; c < c1; c += 8) {
        float u[8];
        int n[8];
#pragma unroll
        for (int i = 0; i < 8; ++i) {
            const bool in = c + i < c1;
            u[i] = in ? a.work[(size_t)(c + i) * all + idx] : 0.f;
            n[i] = in ? a.chunks[2 * (c + i) + 1] : 0;
        }
#pragma unroll
        for (int i = 0; i < 8; ++i) {
            if (c + i >= c1) break;
            a.work[(size_t)(c + i) * all + idx] = S;
            S = fmaf(pw[n[i]], S, u[i]);
        }
    }
    *st = S;
}

// a chunk's outputs: a wave takes 16 of its tokens and the block's value columns, queries and sums in registers
template <typename TI, int DT>
__global__ __launch_bounds__(256) void decayed_chunk_out_kernel(ChunkArgs a) {
    constexpr int KROW = 16 * DT + 4, VT = VBLOCK / 16;
    extern __shared__ __attribute__((aligned(16))) float lds[];
    float* ks = lds;                        // [CHUNK][KROW]
    float* vs = lds + CHUNK * KROW;         // [CHUNK][VROW]
    __shared__ float pw[CHUNK + 1];
    const int c = blockIdx.x, h = blockIdx.y, dv0 = blockIdx.z * VBLOCK;
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, r = lane & 15, grp = lane >> 4;
    const int first = a.chunks[2 * c], rows = a.chunks[2 * c + 1];
    const int D = a.D, Dv = a.Dv, vw = min(VBLOCK, Dv - dv0), vt = (vw + 15) / 16;
    const TI* x = (const TI*)a.x + (size_t)first * a.ldx;
    const int i0 = 16 * wave, row = i0 + r;
    const bool wave_on = i0 < rows, row_ok = row < rows;
    const f32x4 zero = {0.f, 0.f, 0.f, 0.f};

    f32x4 q[DT];
#pragma unroll
    for (int d = 0; d < DT; ++d) {
        const int e = 16 * d + 4 * grp;
        q[d] = row_ok && e < D ? read4(x + (size_t)row * a.ldx + a.q_col + h * D + e) : zero;
    }
    for (int i = threadIdx.x; i <= CHUNK; i += 256) pw[i] = a.powers[(size_t)h * (CHUNK + 1) + i];
    stage_rows<TI>(ks, KROW, x, a.ldx, a.k_col + h * D, D, 16 * DT, rows, a.silu != 0);
    stage_rows<TI>(vs, VROW, x, a.ldx, a.v_col + h * Dv + dv0, vw, 16 * vt, rows, a.silu != 0);
    f32x4 acc[VT];
#pragma unroll
    for (int v = 0; v < VT; ++v) acc[v] = zero;
    if (wave_on) {
#pragma unroll
        for (int d = 0; d < DT; ++d) q[d] = act4(q[d], a.silu != 0);
        // S_0^T q: rows of the state (value columns) from memory, a tile's asked for while the one in front is multiplied
        const float* S = a.work + ((size_t)c * a.H + h) * Dv * D;
        f32x4 s[2][DT];
        auto fetch = [&](int v, f32x4 (&dst)[DT]) {
            const int dv = dv0 + 16 * v + r;
#pragma unroll
            for (int d = 0; d < DT; ++d) {
                const int e = 16 * d + 4 * grp;
                dst[d] = dv < Dv && e < D ? *(const f32x4*)(S + (size_t)dv * D + e) : zero;
            }
        };
        fetch(0, s[0]);
#pragma unroll
        for (int v = 0; v < VT; ++v) {
            if (v < vt) {
                if (v + 1 < vt) fetch(v + 1, s[(v + 1) & 1]);
#pragma unroll
                for (int d = 0; d < DT; ++d)
#pragma unroll
                    for (int k = 0; k < 4; ++k) acc[v] = MFMA_F32(s[v & 1][d][k], q[d][k], acc[v]);
            }
        }
    }
    __syncthreads();
    if (!wave_on) return;
    {
        const float f = pw[min(row + 1, CHUNK)];
#pragma unroll
        for (int v = 0; v < VT; ++v) acc[v] *= f;
    }
    for (int jt = 0; jt <= wave; ++jt) {
        f32x4 p = zero;         // (k_j . q_i): row j = 16 jt + 4 grp + i, column `row`
        const float* kr = ks + (16 * jt + r) * KROW + 4 * grp;
#pragma unroll
        for (int d = 0; d < DT; ++d) {
            const f32x4 kf = *(const f32x4*)(kr + 16 * d);
#pragma unroll
            for (int k = 0; k < 4; ++k) p = MFMA_F32(kf[k], q[d][k], p);
        }
#pragma unroll
        for (int k = 0; k < 4; ++k) {
            const int j = 16 * jt + 4 * grp + k;
            p[k] = j <= row ? p[k] * pw[row - j] : 0.f;
        }
        const float* vr = vs + (16 * jt + 4 * grp) * VROW + r;
#pragma unroll
        for (int v = 0; v < VT; ++v) {
            if (v < vt) {
#pragma unroll
                for (int k = 0; k < 4; ++k) acc[v] = MFMA_F32(vr[k * VROW + 16 * v], p[k], acc[v]);
            }
        }
    }
    // acc[v][i]: value column 16 v + 4 grp + i of token `row`
    if (!row_ok) return;
    float* o = a.o + ((size_t)(first + row) * a.H + h) * Dv + dv0 + 4 * grp;
#pragma unroll
    for (int v = 0; v < VT; ++v)
        if (16 * v + 4 * grp < vw) *(f32x4*)(o + 16 * v) = acc[v];
}

// plan: entries + 1 chunk starts, then n_chunks pairs (first row, rows of at most 64, all of one entry, its chunks in order);
// work: n_chunks * H * Dv * D floats
extern "C" int vt_decayed_attn_chunked(const void* x, int dtype, long long ldx, int q_col, int k_col, int v_col, const float* powers,
                                       float* state, long long slot_stride, const int* plan, const int* slots, float* work,
                                       long long work_floats, float* o, int n_entries, int n_chunks, int H, int D, int Dv, int silu,
                                       hipStream_t stream) {
    VT_REQUIRE(n_entries >= 0 && n_chunks >= n_entries && H > 0 && H <= 65535, "vt_decayed_attn_chunked: bad sizes (%d entries, %d chunks, %d heads)",
               n_entries, n_chunks, H);
    VT_REQUIRE(D > 0 && D <= 256 && D % 4 == 0 && Dv > 0 && Dv % 4 == 0 && Dv <= 65535 * VBLOCK,
               "vt_decayed_attn_chunked: head sizes %d/%d (multiples of 4, keys up to 256)", D, Dv);
    VT_REQUIRE(slot_stride >= (long long)H * D * Dv, "vt_decayed_attn_chunked: state slots are too short");
    VT_REQUIRE(min(q_col, min(k_col, v_col)) >= 0 && ldx >= max(q_col, k_col) + (long long)H * D && ldx >= v_col + (long long)H * Dv,
               "vt_decayed_attn_chunked: rows are too short for their columns");
    VT_REQUIRE(!((ldx | q_col | k_col | v_col) & 3) && !(((uintptr_t)x | (uintptr_t)work | (uintptr_t)o) & 15),
               "vt_decayed_attn_chunked: columns and rows must lie at multiples of 4 elements");
    VT_REQUIRE(work_floats >= (long long)n_chunks * H * D * Dv, "vt_decayed_attn_chunked: %lld floats of scratch memory, %lld needed",
               work_floats, (long long)n_chunks * H * D * Dv);
    const long long blocks = ((long long)H * D * Dv + 255) / 256;
    VT_REQUIRE(blocks <= 0x7fffffff && n_entries <= 65535, "vt_decayed_attn_chunked: too many elements or entries");
    VT_REQUIRE(dtype == VT_F32 || dtype == VT_BF16, "vt_decayed_attn_chunked: unknown dtype %d", dtype);
    if (n_entries == 0) return 0;
    ChunkArgs a;
    a.x = x; a.powers = powers; a.chunk_start = plan; a.chunks = plan + n_entries + 1; a.slots = slots; a.state = state; a.work = work;
    a.o = o; a.ldx = ldx; a.slot_stride = slot_stride; a.q_col = q_col; a.k_col = k_col; a.v_col = v_col; a.H = H; a.D = D; a.Dv = Dv;
    a.silu = silu;
    const dim3 grid(n_chunks, H, (Dv + VBLOCK - 1) / VBLOCK);
#define VT_CHUNKED(KERNEL, TI, DT)                                                                                              \
    do {                                                                                                                        \
        constexpr int bytes = CHUNK * (16 * DT + 4 + VROW) * 4;                                                                 \
        static bool set = false;                                                                                                \
        if (!set) {                                                                                                             \
            hipError_t e = hipFuncSetAttribute((const void*)KERNEL<TI, DT>, hipFuncAttributeMaxDynamicSharedMemorySize, bytes); \
            VT_REQUIRE(e == hipSuccess, "vt_decayed_attn_chunked: cannot get %d bytes of LDS: %s", bytes, hipGetErrorString(e)); \
            set = true;                                                                                                         \
        }                                                                                                                       \
        KERNEL<TI, DT><<<grid, 256, bytes, stream>>>(a);                                                                        \
    } while (0)
#define VT_CHUNKED_DT(KERNEL)                                                                                   \
    do {                                                                                                        \
        if (D <= 16) { if (dtype == VT_F32) VT_CHUNKED(KERNEL, float, 1); else VT_CHUNKED(KERNEL, bf16_t, 1); }        \
        else if (D <= 32) { if (dtype == VT_F32) VT_CHUNKED(KERNEL, float, 2); else VT_CHUNKED(KERNEL, bf16_t, 2); }   \
        else if (D <= 64) { if (dtype == VT_F32) VT_CHUNKED(KERNEL, float, 4); else VT_CHUNKED(KERNEL, bf16_t, 4); }   \
        else if (D <= 128) { if (dtype == VT_F32) VT_CHUNKED(KERNEL, float, 8); else VT_CHUNKED(KERNEL, bf16_t, 8); }  \
        else { if (dtype == VT_F32) VT_CHUNKED(KERNEL, float, 16); else VT_CHUNKED(KERNEL, bf16_t, 16); }              \
    } while (0)
    VT_CHUNKED_DT(decayed_chunk_sum_kernel);
    VT_CHECK_LAUNCH("vt_decayed_attn_chunked(sums)");
    decayed_chunk_state_kernel<<<dim3((unsigned)blocks, n_entries), 256, 0, stream>>>(a);
    VT_CHECK_LAUNCH("vt_decayed_attn_chunked(states)");
    VT_CHUNKED_DT(decayed_chunk_out_kernel);
    VT_CHECK_LAUNCH("vt_decayed_attn_chunked(outputs)");
#undef VT_CHUNKED_DT
#undef VT_CHUNKED
    return 0;
}
