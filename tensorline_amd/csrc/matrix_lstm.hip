// The matrix memory of xLSTM (mLSTM; Beck et al., "xLSTM: Extended Long Short-Term Memory") over a state per head, kept per
// request between steps:
//
//     i_t = cap tanh((gi_t + bi) / cap),  f_t = ln sigmoid(cap tanh((gf_t + bf) / cap)),  m_t = max(f_t + m_(t-1), i_t)
//     S_t = exp(f_t + m_(t-1) - m_t) S_(t-1) + exp(i_t - m_t) k_t v_t^T,   n_t likewise with k_t alone
//     o_t = S_t^T q_t / (max(|n_t . q_t|, exp(-m_t)) + floor)
//
// S, n and m start at zero (the slot is zeroed when it is handed out).  Everything is float.  A slot keeps
// [S: H x dv x dk, transposed: a value column's key rows in a row | n: H x nb x dk | m: H x nb], nb = ceil(dv / 16): every
// block of 16 value columns has a copy of n and m of its own, the same bits in each, so that work-groups that share a head
// read nothing that another of them writes.
//
// Two forms:
//   * tl_mlstm_walk takes the tokens one after another: decode steps and short portions;
//   * tl_mlstm_chunked cuts every sequence's rows of the step into chunks of ML_L tokens.  With F_t the sum of f over the
//     chunk's tokens up to t, g_t = i_t - F_t, G_t the largest g up to t, and S_0, n_0, m_0 what enters the chunk,
//
//       M_t = max(m_0, G_t),  m_t = F_t + M_t,
//       S_t = exp(m_0 - M_t) S_0 + sum_(s <= t) exp(g_s - M_t) k_s v_s^T
//
//     (no exponent is positive), so all but the hand-over from chunk to chunk is independent work:
//       1. mlstm_local_kernel: per chunk and head sum_s exp(g_s - G_L) k_s v_s^T, the same for n, and (F_L, F_L + G_L);
//       2. mlstm_scan_kernel: per state element the chunks of a sequence in order; what enters each chunk replaces the
//          chunk's own term in the workspace, the last state goes to the slot;
//       3. mlstm_outputs_kernel: per chunk and head the L x L matrix exp(g_s - M_t) (q_t . k_s) through LDS, and both
//          products with it and with the entering state.
//     F, g and G are double and only their differences become float, so that a forget gate that closes inside a chunk
//     costs no digits between its neighbours.
//
// Products run on the float matrix instruction (v_mfma_f32_16x16x4_f32).  Lane l = 16 lg + li gives A[li][k] and B[k][li]
// and holds D[4 lg + e][li] in register e; the k of product number v of four is 4 lg + v for both operands.  A state in the
// workspace lies in blocks of 16 key rows x 16 value columns, lane l's four values of a block (rows 4 lg + e, column li)
// next to each other: what kernel 1 holds after its products is what kernel 3 reads as an operand, one kilobyte in a row.
//
// Sums run in a fixed order; the chunked form depends on where a sequence's rows of the step begin, the walk on nothing
// but the sequence: they agree, and agree across cuttings, within rounding.
#include "common.h"

#include <math.h>

#define ML_MAX_DK 256
#define ML_L 64            // tokens per chunk
#define ML_LDP (ML_L + 4)  // floats per LDS row of the [token][token] matrix
#define ML_THREADS 256

typedef float ml_f32x4 __attribute__((ext_vector_type(4)));

// the sum over the 16 lanes of a row, the same bits in each of them
__device__ __forceinline__ float ml_row16_sum(float v) {
#define ML_ROT(N) v += __uint_as_float(__builtin_amdgcn_update_dpp(0, __float_as_uint(v), 0x120 + N, 0xf, 0xf, false))
    ML_ROT(8);
    ML_ROT(4);
    ML_ROT(2);
    ML_ROT(1);
#undef ML_ROT
    return v;
}

__device__ __forceinline__ float ml_dot4(float4 a, float4 b, float s) {
    s = __builtin_fmaf(a.x, b.x, s);
    s = __builtin_fmaf(a.y, b.y, s);
    s = __builtin_fmaf(a.z, b.z, s);
    return __builtin_fmaf(a.w, b.w, s);
}

// four neighbouring values of a row of n from column i on, zeros beyond it
__device__ __forceinline__ float4 ml_load4(const float* __restrict__ row, int i, int n, bool vec) {
    if (vec && i + 4 <= n) return *reinterpret_cast<const float4*>(row + i);
    float4 r;
    r.x = i < n ? row[i] : 0.f;
    r.y = i + 1 < n ? row[i + 1] : 0.f;
    r.z = i + 2 < n ? row[i + 2] : 0.f;
    r.w = i + 3 < n ? row[i + 3] : 0.f;
    return r;
}
__device__ __forceinline__ void ml_store4(float* __restrict__ row, int i, int n, bool vec, float4 v) {
    if (vec && i + 4 <= n) {
        *reinterpret_cast<float4*>(row + i) = v;
        return;
    }
    if (i < n) row[i] = v.x;
    if (i + 1 < n) row[i + 1] = v.y;
    if (i + 2 < n) row[i + 2] = v.z;
    if (i + 3 < n) row[i + 3] = v.w;
}

// the log gates of a token and head from the projections' raw columns
struct MlGates {
    const float *gi, *gf, *bi, *bf;      // [T, >= H] (row strides ldi, ldf), biases [H] or null
    int ldi, ldf;
    float cap;
};
__device__ __forceinline__ float ml_log_input(const MlGates& a, size_t t, int h) {
    return a.cap * tanhf((a.gi[t * a.ldi + h] + (a.bi ? a.bi[h] : 0.f)) / a.cap);
}
__device__ __forceinline__ float ml_log_forget(const MlGates& a, size_t t, int h) {
    const float z = a.cap * tanhf((a.gf[t * a.ldf + h] + (a.bf ? a.bf[h] : 0.f)) / a.cap);
    return fminf(z, 0.f) - log1pf(expf(-fabsf(z)));       // ln sigmoid(z)
}

struct MlState {
    float* base;
    long long stride;
    const int32_t* slots;
};

// ---- token by token -----------------------------------------------------------------------------------------
// A work-group of four waves owns 16 value columns of one head of one sequence, a wave four of them: sixteen lanes share a
// column, each holding 4 M of its rows of S in registers, and as many of n (which every group of sixteen keeps for itself).
template <int M>
__global__ __launch_bounds__(ML_THREADS) void mlstm_walk_kernel(
    const float* __restrict__ q, int ldq, const float* __restrict__ k, int ldk, const float* __restrict__ v, int ldv, MlGates gates,
    float q_scale, float floor_eps, MlState state, const int32_t* __restrict__ q_start, float* __restrict__ out, int ldo, int H, int dk,
    int dv, int vec, int vec_state, int upto) {
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, l = lane & 15;
    const int jb = blockIdx.x, nb = gridDim.x, h = blockIdx.y, s = blockIdx.z;
    const int j = jb * 16 + wave * 4 + (lane >> 4);
    const int r0 = q_start[s], r1 = q_start[s + 1];
    if (r1 <= r0 || r1 - r0 > upto) return;               // the same for the whole work-group
    const bool col_ok = j < dv;
    const int jc = col_ok ? j : dv - 1;
    float* slot = state.base + (size_t)state.slots[s] * state.stride;
    float* st = slot + ((size_t)h * dv + jc) * dk;
    float* np = slot + (size_t)H * dv * dk + ((size_t)h * nb + jb) * dk;
    float* mp = slot + (size_t)H * dv * dk + (size_t)H * nb * dk + (size_t)h * nb + jb;
    const float* qh = q + (size_t)h * dk;
    const float* kh = k + (size_t)h * dk;
    const float* vh = v + (size_t)h * dv + jc;
    float4 S[M], N[M], kc[M], qc[M];
#pragma unroll
    for (int m = 0; m < M; ++m) {
        const int i = (m * 16 + l) * 4;
        S[m] = ml_load4(st, i, dk, vec_state);
        N[m] = ml_load4(np, i, dk, vec_state);
        kc[m] = ml_load4(kh + (size_t)r0 * ldk, i, dk, vec);
        qc[m] = ml_load4(qh + (size_t)r0 * ldq, i, dk, vec);
    }
    float mrun = *mp, vc = vh[(size_t)r0 * ldv];
    for (int t = r0; t < r1; ++t) {
        float4 kn[M], qn[M];
        const int tn = t + 1 < r1 ? t + 1 : t;
#pragma unroll
        for (int m = 0; m < M; ++m) {
            const int i = (m * 16 + l) * 4;
            kn[m] = ml_load4(kh + (size_t)tn * ldk, i, dk, vec);
            qn[m] = ml_load4(qh + (size_t)tn * ldq, i, dk, vec);
        }
        const float vn = vh[(size_t)tn * ldv];
        const float ig = ml_log_input(gates, t, h), fg = ml_log_forget(gates, t, h);
        const float m_new = fmaxf(fg + mrun, ig);
        const float keep = expf(fg + mrun - m_new), add = expf(ig - m_new), av = add * vc;
        mrun = m_new;
        float num = 0.f, den = 0.f;
#pragma unroll
        for (int m = 0; m < M; ++m) {
            S[m].x = __builtin_fmaf(keep, S[m].x, av * kc[m].x);
            S[m].y = __builtin_fmaf(keep, S[m].y, av * kc[m].y);
            S[m].z = __builtin_fmaf(keep, S[m].z, av * kc[m].z);
            S[m].w = __builtin_fmaf(keep, S[m].w, av * kc[m].w);
            N[m].x = __builtin_fmaf(keep, N[m].x, add * kc[m].x);
            N[m].y = __builtin_fmaf(keep, N[m].y, add * kc[m].y);
            N[m].z = __builtin_fmaf(keep, N[m].z, add * kc[m].z);
            N[m].w = __builtin_fmaf(keep, N[m].w, add * kc[m].w);
            num = ml_dot4(S[m], qc[m], num);
            den = ml_dot4(N[m], qc[m], den);
        }
        num = ml_row16_sum(num) * q_scale;
        den = ml_row16_sum(den) * q_scale;
        if (l == 0 && col_ok) out[(size_t)t * ldo + (size_t)h * dv + j] = num / (fmaxf(fabsf(den), expf(-m_new)) + floor_eps);
        vc = vn;
#pragma unroll
        for (int m = 0; m < M; ++m) {
            kc[m] = kn[m];
            qc[m] = qn[m];
        }
    }
    __syncthreads();                                       // every wave has read n and m
#pragma unroll
    for (int m = 0; m < M; ++m) {
        const int i = (m * 16 + l) * 4;
        if (col_ok) ml_store4(st, i, dk, vec_state, S[m]);
        if (threadIdx.x < 16) ml_store4(np, i, dk, vec_state, N[m]);
    }
    if (threadIdx.x == 0) *mp = mrun;
}

// ---- in chunks ------------------------------------------------------------------------------------------------
struct MlChunks {
    const int32_t *seq, *row, *first;    // a chunk's sequence and first row; a sequence's first chunk [S + 1]
};

// F, g = i - F and the running maximum of g for a chunk's n tokens, by the first wave, a token per lane: into LDS, the same
// instructions in both kernels that need them.  Tokens beyond n have g = -infinity.  The caller passes a barrier.
__device__ __forceinline__ void ml_chunk_gates(const MlGates& a, int t0, int n, int h, double* F, double* g, double* G) {
    const int t = threadIdx.x;
    if (t >= ML_L) return;
    double run = t < n ? (double)ml_log_forget(a, t0 + t, h) : 0.0;
#pragma unroll
    for (int off = 1; off < ML_L; off <<= 1) {
        const double below = __shfl_up(run, off, TL_WAVE);
        if (t >= off) run += below;
    }
    const double mine = t < n ? (double)ml_log_input(a, t0 + t, h) - run : -INFINITY;
    double top = mine;
#pragma unroll
    for (int off = 1; off < ML_L; off <<= 1) {
        const double below = __shfl_up(top, off, TL_WAVE);
        if (t >= off) top = fmax(top, below);
    }
    F[t] = run;
    g[t] = mine;
    G[t] = top;
}

// rows t0 .. t0 + n of a [T, ld] matrix, `cols` columns, times `scale`, into LDS rows of `lds_ld` floats; zeros beyond n rows and
// beyond cols up to pad_cols
__device__ __forceinline__ void ml_rows_to_lds(const float* __restrict__ src, int ld, int t0, int n, int cols, int pad_cols, bool vec,
                                               float scale, float* dst, int lds_ld) {
    const int n4 = pad_cols >> 2, total = ML_L * n4;
    for (int base = threadIdx.x; base < total; base += ML_THREADS * 8) {
        float4 r[8];
#pragma unroll
        for (int u = 0; u < 8; ++u) {
            const int idx = base + u * ML_THREADS, tt = idx / n4, i4 = idx - tt * n4;
            r[u] = (idx < total && tt < n) ? ml_load4(src + (size_t)(t0 + tt) * ld, 4 * i4, cols, vec) : make_float4(0.f, 0.f, 0.f, 0.f);
        }
#pragma unroll
        for (int u = 0; u < 8; ++u) {
            const int idx = base + u * ML_THREADS, tt = idx / n4, i4 = idx - tt * n4;
            if (idx < total) {
                r[u].x *= scale, r[u].y *= scale, r[u].z *= scale, r[u].w *= scale;
                *reinterpret_cast<float4*>(dst + tt * lds_ld + 4 * i4) = r[u];
            }
        }
    }
}

// Grid (chunk, head, groups of 8 blocks of value columns); wave w takes blocks w and w + 4 of its group.
__global__ __launch_bounds__(ML_THREADS) void mlstm_local_kernel(
    const float* __restrict__ k, int ldk, const float* __restrict__ v, int ldv, MlGates gates, MlState state, MlChunks chunks,
    const int32_t* __restrict__ q_start, float* __restrict__ ws_s, float* __restrict__ ws_n, double* __restrict__ ws_g,
    float* __restrict__ ws_m, int H, int dk, int dv, int vec) {
    extern __shared__ __attribute__((aligned(16))) float ml_smem[];
    __shared__ double F[ML_L], g[ML_L], G[ML_L];
    __shared__ float w[ML_L];
    const int c = blockIdx.x, h = blockIdx.y, tid = threadIdx.x;
    const int s = chunks.seq[c], t0 = chunks.row[c];
    const int n = min(ML_L, q_start[s + 1] - t0);
    const int DKP = (dk + 15) & ~15, LD = DKP + 4, nb = (dv + 15) >> 4, kb = DKP >> 4;
    const int lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), li = lane & 15, lg = lane >> 4;
    const int jb0 = blockIdx.z * 8 + wave;
    const float* vb = v + (size_t)t0 * ldv + (size_t)h * dv;
    float bf[2][4][4];                                     // B: values (asked for ahead of all else), token 16 sb + 4 lg + e, column li
#pragma unroll
    for (int u = 0; u < 2; ++u)
#pragma unroll
        for (int sb = 0; sb < 4; ++sb)
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                const int t = 16 * sb + 4 * lg + e, j = (jb0 + 4 * u) * 16 + li;
                bf[u][sb][e] = t < n && j < dv ? vb[(uint32_t)(t * ldv + j)] : 0.f;
            }
    float* Ks = ml_smem;
    ml_rows_to_lds(k + (size_t)h * dk, ldk, t0, n, dk, DKP, vec, 1.0f, Ks, LD);
    ml_chunk_gates(gates, t0, n, h, F, g, G);
    __syncthreads();
    if (tid < ML_L) w[tid] = tid < n ? expf((float)(g[tid] - G[ML_L - 1])) : 0.f;
    const size_t at = (size_t)c * H + h;
    if (blockIdx.z == 0 && tid == 0) {
        ws_g[2 * at] = F[ML_L - 1];
        ws_g[2 * at + 1] = F[ML_L - 1] + G[ML_L - 1];
        // what enters a sequence's first chunk, for the scan (which overwrites the slot)
        if (c == chunks.first[s])
            ws_m[at] = state.base[(size_t)state.slots[s] * state.stride + (size_t)H * dv * dk + (size_t)H * nb * dk + (size_t)h * nb];
    }
    __syncthreads();
    if (blockIdx.z == 0) {
        for (int i = tid; i < DKP; i += ML_THREADS) {
            float sum = 0.f;
#pragma unroll 16
            for (int t = 0; t < ML_L; ++t) sum = __builtin_fmaf(w[t], Ks[t * LD + i], sum);
            ws_n[at * DKP + i] = sum;
        }
    }
    if (jb0 >= nb) return;                                 // no barrier follows
    const bool two = jb0 + 4 < nb;
#pragma unroll
    for (int sb = 0; sb < 4; ++sb)
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            const float we = w[16 * sb + 4 * lg + e];
            bf[0][sb][e] *= we;
            bf[1][sb][e] *= we;
        }
    float* dst = ws_s + at * (size_t)kb * nb * 256;
    for (int ib = 0; ib < kb; ++ib) {
        ml_f32x4 acc0 = {0.f, 0.f, 0.f, 0.f}, acc1 = {0.f, 0.f, 0.f, 0.f};
        const float* kr = Ks + 4 * lg * LD + ib * 16 + li;
#pragma unroll
        for (int sb = 0; sb < 4; ++sb)
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                const float a = kr[(16 * sb + e) * LD];
                acc0 = __builtin_amdgcn_mfma_f32_16x16x4f32(a, bf[0][sb][e], acc0, 0, 0, 0);
                if (two) acc1 = __builtin_amdgcn_mfma_f32_16x16x4f32(a, bf[1][sb][e], acc1, 0, 0, 0);
            }
        *reinterpret_cast<ml_f32x4*>(dst + ((size_t)(ib * nb + jb0) * 64 + lane) * 4) = acc0;
        if (two) *reinterpret_cast<ml_f32x4*>(dst + ((size_t)(ib * nb + jb0 + 4) * 64 + lane) * 4) = acc1;
    }
}

#define ML_RING 4       // fragments of the entering state on their way
#define ML_AHEAD 4      // chunks whose terms are on their way while the ones before are added
// Grid (quadruples of state elements / 256, then one block for n; head; sequence).
__global__ __launch_bounds__(ML_THREADS) void mlstm_scan_kernel(float* __restrict__ ws_s, float* __restrict__ ws_n,
                                                                const double* __restrict__ ws_g, float* __restrict__ ws_m,
                                                                MlState state, MlChunks chunks, int H, int dk, int dv, int s_blocks,
                                                                int vec_state) {
    const int h = blockIdx.y, s = blockIdx.z, tid = threadIdx.x;
    const int c0 = chunks.first[s], c1 = chunks.first[s + 1];
    if (c1 <= c0) return;
    const int DKP = (dk + 15) & ~15, nb = (dv + 15) >> 4, kb = DKP >> 4;
    float* slot = state.base + (size_t)state.slots[s] * state.stride;
    float m = ws_m[(size_t)c0 * H + h];
    auto step = [&](int c, float& keep, float& add) {      // the factors on what enters chunk c and on its own term; m moves on
        const double Fl = ws_g[2 * ((size_t)c * H + h)], ml = ws_g[2 * ((size_t)c * H + h) + 1];
        const float m_new = (float)fmax(Fl + (double)m, ml);
        keep = expf((float)(Fl + (double)m - (double)m_new));
        add = expf((float)(ml - (double)m_new));
        m = m_new;
    };
    if ((int)blockIdx.x >= s_blocks) {                     // n and m
        float* ncopies = slot + (size_t)H * dv * dk + (size_t)h * nb * dk;
        const int i = tid;
        const bool mine = i < DKP;
        float N = (mine && i < dk) ? ncopies[i] : 0.f;
        for (int c = c0; c < c1; ++c) {
            const size_t at = (size_t)c * H + h;
            if (tid == 0 && c > c0) ws_m[at] = m;
            float keep, add;
            step(c, keep, add);
            if (mine) {
                const float local = ws_n[at * DKP + i];
                ws_n[at * DKP + i] = N;
                N = __builtin_fmaf(keep, N, add * local);
            }
        }
        if (mine && i < dk)
            for (int b = 0; b < nb; ++b) ncopies[(size_t)b * dk + i] = N;
        if (tid < nb) slot[(size_t)H * dv * dk + (size_t)H * nb * dk + (size_t)h * nb + tid] = m;
        for (int b = tid + ML_THREADS; b < nb; b += ML_THREADS) slot[(size_t)H * dv * dk + (size_t)H * nb * dk + (size_t)h * nb + b] = m;
        return;
    }
    const int e = blockIdx.x * ML_THREADS + tid;
    if (e >= kb * nb * 64) return;
    const int blk = e >> 6, lane = e & 63, ib = blk / nb, jb = blk - ib * nb;
    const int i = ib * 16 + 4 * (lane >> 4), j = jb * 16 + (lane & 15);
    float* st = slot + ((size_t)h * dv + (j < dv ? j : dv - 1)) * dk;
    float4 S = j < dv ? ml_load4(st, i, dk, vec_state) : make_float4(0.f, 0.f, 0.f, 0.f);
    const size_t per = (size_t)kb * nb * 64;               // quadruples of a chunk and head
    float4* w4 = reinterpret_cast<float4*>(ws_s) + e;
    for (int cb = c0; cb < c1; cb += ML_AHEAD) {
        float4 local[ML_AHEAD];
#pragma unroll
        for (int u = 0; u < ML_AHEAD; ++u) local[u] = w4[((size_t)min(cb + u, c1 - 1) * H + h) * per];
#pragma unroll
        for (int u = 0; u < ML_AHEAD; ++u) {
            if (cb + u >= c1) break;
            float keep, add;
            step(cb + u, keep, add);
            w4[((size_t)(cb + u) * H + h) * per] = S;
            S.x = __builtin_fmaf(keep, S.x, add * local[u].x);
            S.y = __builtin_fmaf(keep, S.y, add * local[u].y);
            S.z = __builtin_fmaf(keep, S.z, add * local[u].z);
            S.w = __builtin_fmaf(keep, S.w, add * local[u].w);
        }
    }
    if (j < dv) ml_store4(st, i, dk, vec_state, S);
}

// Grid (chunk, head, z): z takes groups z, z + gridDim.z, .. of 8 blocks of value columns.  First wave w takes tokens 16 w .. of the matrix (which every
// work-group computes for itself), then blocks w and w + 4 of each of its groups.
__global__ __launch_bounds__(ML_THREADS, 2) void mlstm_outputs_kernel(
    const float* __restrict__ q, int ldq, const float* __restrict__ k, int ldk, const float* __restrict__ v, int ldv, MlGates gates,
    float q_scale, float floor_eps, MlChunks chunks, const int32_t* __restrict__ q_start, const float* __restrict__ ws_s,
    const float* __restrict__ ws_n, const float* __restrict__ ws_m, float* __restrict__ out, int ldo, int H, int dk, int dv, int vec) {
    extern __shared__ __attribute__((aligned(16))) float ml_smem[];
    __shared__ double F[ML_L], g[ML_L], G[ML_L];
    __shared__ float into[ML_L], nq[ML_L], den[ML_L];
    const int c = blockIdx.x, h = blockIdx.y, tid = threadIdx.x;
    const int s = chunks.seq[c], t0 = chunks.row[c];
    const int n = min(ML_L, q_start[s + 1] - t0);
    const int DKP = (dk + 15) & ~15, LD = DKP + 4, nb = (dv + 15) >> 4, kb = DKP >> 4;
    const size_t at = (size_t)c * H + h;
    float* Qs = ml_smem;                                   // [L][LD]
    float* Ks = Qs + ML_L * LD;                            // [L][LD], later
    float* Ps = Ks;                                        // [L][ML_LDP]: exp(g_s - M_t) (q_t . k_s), s <= t
    ml_rows_to_lds(q + (size_t)h * dk, ldq, t0, n, dk, DKP, vec, q_scale, Qs, LD);
    ml_rows_to_lds(k + (size_t)h * dk, ldk, t0, n, dk, DKP, vec, 1.0f, Ks, LD);
    ml_chunk_gates(gates, t0, n, h, F, g, G);
    const double m0 = (double)ws_m[at];
    __syncthreads();
    if (tid < ML_L) {
        const double M = fmax(m0, G[tid]);
        G[tid] = M;                                        // from here on M_t
        into[tid] = expf((float)(m0 - M));
    }
    const int lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), li = lane & 15, lg = lane >> 4;
    {
        // n_0 . q_t: four lanes to a token
        const int t = tid >> 2, part = tid & 3;
        const float* n0 = ws_n + at * DKP;
        float sum = 0.f;
        for (int i = 4 * part; i < DKP; i += 16)
            sum = ml_dot4(*reinterpret_cast<const float4*>(n0 + i), *reinterpret_cast<const float4*>(Qs + t * LD + i), sum);
        sum += __shfl_xor(sum, 1, TL_WAVE);
        sum += __shfl_xor(sum, 2, TL_WAVE);
        if (part == 0) nq[t] = sum;
    }
    ml_f32x4 acc[4];
#pragma unroll
    for (int sb = 0; sb < 4; ++sb) acc[sb] = ml_f32x4{0.f, 0.f, 0.f, 0.f};
    for (int ib = 0; ib < kb; ++ib) {
        const float4 a = *reinterpret_cast<const float4*>(Qs + (wave * 16 + li) * LD + ib * 16 + 4 * lg);
        float4 b[4];
#pragma unroll
        for (int sb = 0; sb < 4; ++sb)
            if (sb <= wave) b[sb] = *reinterpret_cast<const float4*>(Ks + (sb * 16 + li) * LD + ib * 16 + 4 * lg);
#define ML_EACH(X)                                                                                             \
    _Pragma("unroll") for (int sb = 0; sb < 4; ++sb)                                                           \
        if (sb <= wave) acc[sb] = __builtin_amdgcn_mfma_f32_16x16x4f32(a.X, b[sb].X, acc[sb], 0, 0, 0);
        ML_EACH(x)
        ML_EACH(y)
        ML_EACH(z)
        ML_EACH(w)
#undef ML_EACH
    }
    // What the second half needs from memory is asked for here, ahead of the barriers: the values of this wave's first two blocks
    // of columns and the first of the entering state's fragments.
    const float4* S0 = reinterpret_cast<const float4*>(ws_s + at * (size_t)kb * nb * 256);
    const float* vb = v + (size_t)t0 * ldv + (size_t)h * dv;
    float bv[2][4][4];                                     // B of the second product: token 16 sb + 4 lg + e, column li
    float4 ring[ML_RING][2];
    int jb0 = blockIdx.z * 8 + wave;
    auto fetch = [&]() {
#pragma unroll
        for (int r = 0; r < ML_RING; ++r)
#pragma unroll
            for (int u = 0; u < 2; ++u)
                ring[r][u] = S0[(uint32_t)((min(r, kb - 1) * nb + min(jb0 + 4 * u, nb - 1)) * 64 + lane)];
#pragma unroll
        for (int u = 0; u < 2; ++u)
#pragma unroll
            for (int sb = 0; sb < 4; ++sb)
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    // (beyond the chunk's tokens the matrix is zero, beyond dv nothing is written: any finite value will do)
                    const int t = min(16 * sb + 4 * lg + e, n - 1), j = min((jb0 + 4 * u) * 16 + li, dv - 1);
                    bv[u][sb][e] = vb[(uint32_t)(t * ldv + j)];
                }
    };
    fetch();
    __syncthreads();                                       // the keys are done with; M, into and nq are there
    {
        // this lane holds tokens t = 16 wave + 4 lg + e and s = 16 sb + li
        float rows[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int sb = 0; sb < 4; ++sb)
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                const int t = wave * 16 + 4 * lg + e, ss = sb * 16 + li;
                const float p = (sb <= wave && ss <= t && t < n) ? acc[sb][e] * expf((float)(g[ss] - G[t])) : 0.f;
                Ps[t * ML_LDP + ss] = p;
                rows[e] += p;
            }
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            const int t = wave * 16 + 4 * lg + e;
            const float sum = ml_row16_sum(rows[e]) + into[t] * nq[t];
            if (li == 0) den[t] = 1.0f / (fmaxf(fabsf(sum), expf((float)-(F[t] + G[t]))) + floor_eps);
        }
    }
    __syncthreads();
    for (; jb0 < nb; jb0 += 8 * gridDim.z) {               // no barrier in here
        const bool two = jb0 + 4 < nb;
        const int jb1 = jb0 + 4;
        ml_f32x4 y[4][2];
#pragma unroll
        for (int tb = 0; tb < 4; ++tb) y[tb][0] = y[tb][1] = ml_f32x4{0.f, 0.f, 0.f, 0.f};
        for (int base = 0; base < kb; base += ML_RING) {
#pragma unroll
            for (int r = 0; r < ML_RING; ++r) {
                const int ib = base + r;
                if (ib >= kb) break;
                const float4 s0 = ring[r][0], s1 = ring[r][1];
                // the place in the ring is taken by the fragment ML_RING steps further on
                if (ib + ML_RING < kb) {
                    ring[r][0] = S0[(uint32_t)(((ib + ML_RING) * nb + jb0) * 64 + lane)];
                    ring[r][1] = S0[(uint32_t)(((ib + ML_RING) * nb + min(jb1, nb - 1)) * 64 + lane)];
                }
                float4 a[4];
#pragma unroll
                for (int tb = 0; tb < 4; ++tb) a[tb] = *reinterpret_cast<const float4*>(Qs + (tb * 16 + li) * LD + ib * 16 + 4 * lg);
#define ML_EACH(X)                                                                                             \
    _Pragma("unroll") for (int tb = 0; tb < 4; ++tb) {                                                         \
        y[tb][0] = __builtin_amdgcn_mfma_f32_16x16x4f32(a[tb].X, s0.X, y[tb][0], 0, 0, 0);                     \
        if (two) y[tb][1] = __builtin_amdgcn_mfma_f32_16x16x4f32(a[tb].X, s1.X, y[tb][1], 0, 0, 0);            \
    }
                ML_EACH(x)
                ML_EACH(y)
                ML_EACH(z)
                ML_EACH(w)
#undef ML_EACH
                __builtin_amdgcn_sched_barrier(0);           // reads of later steps stay there: registers
            }
        }
#pragma unroll
        for (int tb = 0; tb < 4; ++tb)
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                const float f = into[tb * 16 + 4 * lg + e];
                y[tb][0][e] *= f;
                y[tb][1][e] *= f;
            }
#pragma unroll
        for (int sb = 0; sb < 4; ++sb) {
            float4 a[4];
#pragma unroll
            for (int tb = sb; tb < 4; ++tb) a[tb] = *reinterpret_cast<const float4*>(Ps + (tb * 16 + li) * ML_LDP + sb * 16 + 4 * lg);
#define ML_EACH(X, E)                                                                                          \
    _Pragma("unroll") for (int tb = sb; tb < 4; ++tb) {                                                        \
        y[tb][0] = __builtin_amdgcn_mfma_f32_16x16x4f32(a[tb].X, bv[0][sb][E], y[tb][0], 0, 0, 0);             \
        if (two) y[tb][1] = __builtin_amdgcn_mfma_f32_16x16x4f32(a[tb].X, bv[1][sb][E], y[tb][1], 0, 0, 0);    \
    }
            ML_EACH(x, 0)
            ML_EACH(y, 1)
            ML_EACH(z, 2)
            ML_EACH(w, 3)
#undef ML_EACH
            __builtin_amdgcn_sched_barrier(0);
        }
        // this lane holds tokens t = 16 tb + 4 lg + e and value column 16 jb + li
#pragma unroll
        for (int tb = 0; tb < 4; ++tb)
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                const int t = tb * 16 + 4 * lg + e;
                if (t >= n) continue;
                const float d = den[t];
                float* o = out + (size_t)(t0 + t) * ldo + (size_t)h * dv;
                if (jb0 * 16 + li < dv) o[jb0 * 16 + li] = y[tb][0][e] * d;
                if (two && jb1 * 16 + li < dv) o[jb1 * 16 + li] = y[tb][1][e] * d;
            }
        if (jb0 + 8 * (int)gridDim.z < nb) {               // the next blocks' values and fragments
            jb0 += 8 * gridDim.z;
            fetch();
            jb0 -= 8 * gridDim.z;
        }
    }
}

extern "C" int tl_mlstm_takes(int dk, int dv) { return dk > 0 && dk <= ML_MAX_DK && dv > 0; }
// floats of a request's state
extern "C" long long tl_mlstm_state_floats(int H, int dk, int dv) {
    const long long nb = (dv + 15) / 16;
    return (long long)H * ((long long)dv * dk + nb * (dk + 1));
}
// floats of the workspace per chunk and head: the state in blocks, then n
extern "C" long long tl_mlstm_workspace(int dk, int dv) {
    const long long kb = (dk + 15) / 16, nb = (dv + 15) / 16;
    return kb * nb * 256 + kb * 16;
}

static int ml_check(const char* who, const float* q, int ldq, const float* k, int ldk, const float* v, int ldv, const MlGates& a,
                    long long state_stride, int S, int H, int dk, int dv, int ldo) {
    TL_CHECK_ARG(S >= 0 && H > 0 && tl_mlstm_takes(dk, dv), "%s: bad sizes H=%d dk=%d dv=%d", who, H, dk, dv);
    TL_CHECK_ARG(ldq >= H * dk && ldk >= H * dk && ldv >= H * dv && ldo >= H * dv && a.ldi >= H && a.ldf >= H, "%s: rows too short", who);
    TL_CHECK_ARG(q && k && v && a.gi && a.gf && a.cap > 0.f, "%s: operands are missing or the gates' cap %g is not positive", who, (double)a.cap);
    TL_CHECK_ARG(state_stride >= tl_mlstm_state_floats(H, dk, dv), "%s: the state of a request is too small", who);
    TL_CHECK_ARG(S <= 65535 && H <= 65535, "%s: too many sequences or heads for one launch", who);
    return 0;
}
static int ml_vec(const float* q, int ldq, const float* k, int ldk, int dk) {
    return ((uintptr_t)q % 16 == 0 && (uintptr_t)k % 16 == 0 && ldq % 4 == 0 && ldk % 4 == 0 && dk % 4 == 0) ? 1 : 0;
}
static int ml_vec_state(const float* state, long long stride, int dk) {
    return ((uintptr_t)state % 16 == 0 && stride % 4 == 0 && dk % 4 == 0) ? 1 : 0;
}

// q, k [T, >= H * dk], v [T, >= H * dv], gi, gf [T, >= H] raw gate columns, bi, bf [H] or null; state: see the head of the
// file; sequences that bring more than `upto` tokens are left alone (upto 0: none is).
extern "C" int tl_mlstm_walk(const float* q, int ldq, const float* k, int ldk, const float* v, int ldv, const float* gi, int ldi,
                             const float* gf, int ldf, const float* bi, const float* bf, float cap, float q_scale, float floor_eps,
                             float* state, long long state_stride, const int32_t* state_slots, const int32_t* q_start, float* out,
                             int ldo, int S, int H, int dk, int dv, int upto, hipStream_t stream) {
    const MlGates a{gi, gf, bi, bf, ldi, ldf, cap};
    if (int rc = ml_check("tl_mlstm_walk", q, ldq, k, ldk, v, ldv, a, state_stride, S, H, dk, dv, ldo)) return rc;
    if (S == 0) return 0;
    const MlState st{state, state_stride, state_slots};
    const int vec = ml_vec(q, ldq, k, ldk, dk), vs = ml_vec_state(state, state_stride, dk);
    const int most = upto > 0 ? upto : 0x7fffffff;
    dim3 grid((dv + 15) / 16, H, S), block(ML_THREADS);
#define GO(MV)                                                                                                          \
    hipLaunchKernelGGL(mlstm_walk_kernel<MV>, grid, block, 0, stream, q, ldq, k, ldk, v, ldv, a, q_scale, floor_eps, st, q_start, \
                       out, ldo, H, dk, dv, vec, vs, most)
    if (dk <= 64) GO(1);
    else if (dk <= 128) GO(2);
    else if (dk <= 192) GO(3);
    else GO(4);
#undef GO
    TL_CHECK_LAUNCH("tl_mlstm_walk");
    return 0;
}

// The same operands; chunk_seq, chunk_row [chunks], chunk_first [S + 1]; ws: chunks * H * tl_mlstm_workspace floats (16-byte
// aligned), ws_g: chunks * H * 2 doubles, ws_m: chunks * H floats.  Sequences without chunks are left alone.
extern "C" int tl_mlstm_chunked(const float* q, int ldq, const float* k, int ldk, const float* v, int ldv, const float* gi, int ldi,
                                const float* gf, int ldf, const float* bi, const float* bf, float cap, float q_scale, float floor_eps,
                                float* state, long long state_stride, const int32_t* state_slots, const int32_t* q_start,
                                const int32_t* chunk_seq, const int32_t* chunk_row, const int32_t* chunk_first, float* ws, double* ws_g,
                                float* ws_m, float* out, int ldo, int S, int chunks, int H, int dk, int dv, hipStream_t stream) {
    const MlGates a{gi, gf, bi, bf, ldi, ldf, cap};
    if (int rc = ml_check("tl_mlstm_chunked", q, ldq, k, ldk, v, ldv, a, state_stride, S, H, dk, dv, ldo)) return rc;
    TL_CHECK_ARG(ws && ws_g && ws_m && (uintptr_t)ws % 16 == 0 && (uintptr_t)ws_g % 8 == 0, "tl_mlstm_chunked: the (16-byte aligned) workspace is missing");
    TL_CHECK_ARG((long long)ML_L * ldv < (1ll << 31), "tl_mlstm_chunked: rows of %d values are too long", ldv);
    TL_CHECK_ARG(chunk_seq && chunk_row && chunk_first && chunks >= 0, "tl_mlstm_chunked: chunk tables are missing");
    if (S == 0 || chunks == 0) return 0;
    const MlState st{state, state_stride, state_slots};
    const MlChunks ch{chunk_seq, chunk_row, chunk_first};
    const int vec = ml_vec(q, ldq, k, ldk, dk), vs = ml_vec_state(state, state_stride, dk);
    const int DKP = (dk + 15) / 16 * 16, nb = (dv + 15) / 16, kb = DKP / 16;
    float* ws_n = ws + (size_t)chunks * H * kb * nb * 256;
    const size_t rows = sizeof(float) * ML_L * (DKP + 4);
    const size_t pbytes = sizeof(float) * ML_L * ML_LDP;
    const size_t lds_c = rows + (rows > pbytes ? rows : pbytes);
    TL_CHECK_ARG(lds_c <= 150 * 1024, "tl_mlstm_chunked: a key size of %d needs %zu bytes of LDS", dk, lds_c);
    TL_CHECK_ARG((nb + 7) / 8 <= 65535, "tl_mlstm_chunked: a value size of %d is more than a launch takes", dv);
    hipLaunchKernelGGL(mlstm_local_kernel, dim3(chunks, H, (nb + 7) / 8), dim3(ML_THREADS), rows, stream, k, ldk, v, ldv, a, st, ch, q_start,
                       ws, ws_n, ws_g, ws_m, H, dk, dv, vec);
    TL_CHECK_LAUNCH("tl_mlstm_chunked local states");
    const int s_blocks = tl_ceil_div(kb * nb * 64, ML_THREADS);
    hipLaunchKernelGGL(mlstm_scan_kernel, dim3(s_blocks + 1, H, S), dim3(ML_THREADS), 0, stream, ws, ws_n, ws_g, ws_m, st, ch, H, dk, dv,
                       s_blocks, vs);
    TL_CHECK_LAUNCH("tl_mlstm_chunked scan");
    // few chunks and heads: the groups of value columns to work-groups of their own; many: one after another in one
    const int groups = (long long)chunks * H < 512 ? (nb + 7) / 8 : 1;
    hipLaunchKernelGGL(mlstm_outputs_kernel, dim3(chunks, H, groups), dim3(ML_THREADS), lds_c, stream, q, ldq, k, ldk, v, ldv, a, q_scale, floor_eps,
                       ch, q_start, ws, ws_n, ws_m, out, ldo, H, dk, dv, vec);
    TL_CHECK_LAUNCH("tl_mlstm_chunked outputs");
    return 0;
}
