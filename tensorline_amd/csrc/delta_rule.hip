// The gated delta rule over a matrix state per head, kept per request between steps:
//
//     S <- g_t S;   u_t = beta_t (v_t - S^T k_t);   S <- S + k_t u_t^T;   o_t = S^T q_t
//
// with beta_t = sigmoid(b_t) and g_t = exp(-exp(rate_log) softplus(a_t + step_bias)), one of each per token and head.
// Queries and keys come as they enter the rule (unit vectors, scaled), shared by the `share` consecutive value heads of a
// group.  Everything is float; S of a head is kept transposed in the slot, [value column][key row].
//
// Two forms:
//   * tl_delta_walk takes the tokens one after another: decode steps and short portions.
//   * tl_delta_chunked cuts every sequence's rows of the step into chunks of DR_L tokens (Yang, Wang, Zhang, Shen and Kim,
//     "Parallelizing Linear Transformers with the Delta Rule over Sequence Length"; with decays: Yang, Kautz and
//     Hatamizadeh, "Gated Delta Networks: Improving Mamba2 with Delta Rule").  With c_t the sum of ln g over the chunk's
//     tokens up to t and S_0 the state that enters the chunk,
//
//       u_t = beta_t (v_t - exp(c_t) S_0^T k_t - sum_(s < t) exp(c_t - c_s) (k_t . k_s) u_s)
//
//     is a triangular system (I + A) U = diag(beta) (V - diag(exp c) K S_0), A_ts = beta_t exp(c_t - c_s) (k_t . k_s):
//       1. delta_prepare_kernel solves it for both right-hand sides, U_0 = (I + A)^-1 diag(beta) V and W = (I + A)^-1
//          diag(beta exp c) K, per chunk and head, all chunks at once;
//       2. delta_states_kernel walks the chunks of a sequence: U = U_0 - W S_0, S_L = exp(c_L) S_0 + sum_s exp(c_L - c_s)
//          k_s u_s^T, a work-group per head and 16 value columns, leaving U and every chunk's S_0 in the workspace;
//       3. delta_outputs_kernel: o_t = exp(c_t) S_0^T q_t + sum_(s <= t) exp(c_t - c_s) (q_t . k_s) u_s, all chunks at once.
//     The sums c are double and only their differences (never positive) become float, so that a chunk of strong decays
//     costs no digits between weak ones.  Products run on the float matrix instruction (v_mfma_f32_16x16x4_f32).
//
// Sums run in a fixed order; the chunked form depends on where a sequence's rows of the step begin, the walk on nothing
// but the sequence: they agree, and agree across cuttings, within rounding.
#include "common.h"

#include <math.h>

#define DR_MAX_DK 256      // the walk's largest key size
#define DR_L 64            // tokens per chunk
#define DR_LDA (DR_L + 4)  // floats per LDS row of a [token][token] matrix
#define DR_THREADS 256

typedef float dr_f32x4 __attribute__((ext_vector_type(4)));

__device__ __forceinline__ float dr_softplus(float z) { return fmaxf(z, 0.f) + log1pf(expf(-fabsf(z))); }
__device__ __forceinline__ float dr_sigmoid(float z) { return 1.0f / (1.0f + expf(-z)); }

// the sum over the 16 lanes of a row, the same bits in each of them
__device__ __forceinline__ float dr_row16_sum(float v) {
#define DR_ROT(N) v += __uint_as_float(__builtin_amdgcn_update_dpp(0, __float_as_uint(v), 0x120 + N, 0xf, 0xf, false))
    DR_ROT(8);
    DR_ROT(4);
    DR_ROT(2);
    DR_ROT(1);
#undef DR_ROT
    return v;
}

__device__ __forceinline__ float dr_dot4(float4 a, float4 b, float s) {
    s = __builtin_fmaf(a.x, b.x, s);
    s = __builtin_fmaf(a.y, b.y, s);
    s = __builtin_fmaf(a.z, b.z, s);
    return __builtin_fmaf(a.w, b.w, s);
}

// four neighbouring values of a row of n from column i on, zeros beyond it
__device__ __forceinline__ float4 dr_load4(const float* __restrict__ row, int i, int n, bool vec) {
    if (vec && i + 4 <= n) return *reinterpret_cast<const float4*>(row + i);
    float4 r;
    r.x = i < n ? row[i] : 0.f;
    r.y = i + 1 < n ? row[i + 1] : 0.f;
    r.z = i + 2 < n ? row[i + 2] : 0.f;
    r.w = i + 3 < n ? row[i + 3] : 0.f;
    return r;
}
__device__ __forceinline__ void dr_store4(float* __restrict__ row, int i, int n, bool vec, float4 v) {
    if (vec && i + 4 <= n) {
        *reinterpret_cast<float4*>(row + i) = v;
        return;
    }
    if (i < n) row[i] = v.x;
    if (i + 1 < n) row[i + 1] = v.y;
    if (i + 2 < n) row[i + 2] = v.z;
    if (i + 3 < n) row[i + 3] = v.w;
}

// ---- token by token -----------------------------------------------------------------------------------------
// A work-group of four waves owns 16 value columns of one head of one sequence, a wave four of them: sixteen lanes share
// a column, each holding 4 M of its rows of S in registers, and put their shares of S^T k, S^T q and k . q together by
// lane rotations: a token costs no barrier.  The state before the update gives the output too:
// o = g S^T q + (k . q) u.  The next token's operands are on their way meanwhile.
template <int M>
__global__ __launch_bounds__(DR_THREADS) void delta_walk_kernel(
    const float* __restrict__ q, int ldq, const float* __restrict__ k, int ldk, const float* __restrict__ v, int ldv,
    const float* __restrict__ b, int ldb, const float* __restrict__ a, int lda, const float* __restrict__ rate_log,
    const float* __restrict__ step_bias, int share, float* __restrict__ state, long long state_stride,
    const int32_t* __restrict__ state_slots, const int32_t* __restrict__ q_start, float* __restrict__ out, int ldo, int dk,
    int dv, int vec, int vec_state) {
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, l = lane & 15;
    const int j = blockIdx.x * 16 + wave * 4 + (lane >> 4), h = blockIdx.y, s = blockIdx.z;
    const int r0 = q_start[s], r1 = q_start[s + 1];
    if (r1 <= r0) return;
    const bool col_ok = j < dv;
    const int jc = col_ok ? j : dv - 1;
    float* st = state + (size_t)state_slots[s] * state_stride + ((size_t)h * dv + jc) * dk;
    const float* qh = q + (size_t)(h / share) * dk;
    const float* kh = k + (size_t)(h / share) * dk;
    const float* vh = v + (size_t)h * dv + jc;
    const float rate = expf(rate_log[h]), bias = step_bias ? step_bias[h] : 0.f;
    float4 S[M], kc[M], qc[M];
#pragma unroll
    for (int m = 0; m < M; ++m) {
        const int i = (m * 16 + l) * 4;
        S[m] = dr_load4(st, i, dk, vec_state);
        kc[m] = dr_load4(kh + (size_t)r0 * ldk, i, dk, vec);
        qc[m] = dr_load4(qh + (size_t)r0 * ldq, i, dk, vec);
    }
    float vc = vh[(size_t)r0 * ldv], bc = b[(size_t)r0 * ldb + h], ac = a[(size_t)r0 * lda + h];
    for (int t = r0; t < r1; ++t) {
        float4 kn[M], qn[M];
        const int tn = t + 1 < r1 ? t + 1 : t;
#pragma unroll
        for (int m = 0; m < M; ++m) {
            const int i = (m * 16 + l) * 4;
            kn[m] = dr_load4(kh + (size_t)tn * ldk, i, dk, vec);
            qn[m] = dr_load4(qh + (size_t)tn * ldq, i, dk, vec);
        }
        const float vn = vh[(size_t)tn * ldv], bn = b[(size_t)tn * ldb + h], an = a[(size_t)tn * lda + h];
        const float beta = dr_sigmoid(bc), g = expf(-rate * dr_softplus(ac + bias));
        float sk = 0.f, sq = 0.f, kq = 0.f;
#pragma unroll
        for (int m = 0; m < M; ++m) {
            sk = dr_dot4(S[m], kc[m], sk);
            sq = dr_dot4(S[m], qc[m], sq);
            kq = dr_dot4(kc[m], qc[m], kq);
        }
        sk = dr_row16_sum(sk);
        sq = dr_row16_sum(sq);
        kq = dr_row16_sum(kq);
        const float u = beta * (vc - g * sk);
        if (l == 0 && col_ok) out[(size_t)t * ldo + (size_t)h * dv + j] = __builtin_fmaf(kq, u, g * sq);
#pragma unroll
        for (int m = 0; m < M; ++m) {
            S[m].x = __builtin_fmaf(kc[m].x, u, g * S[m].x);
            S[m].y = __builtin_fmaf(kc[m].y, u, g * S[m].y);
            S[m].z = __builtin_fmaf(kc[m].z, u, g * S[m].z);
            S[m].w = __builtin_fmaf(kc[m].w, u, g * S[m].w);
            kc[m] = kn[m];
            qc[m] = qn[m];
        }
        vc = vn, bc = bn, ac = an;
    }
    if (col_ok) {
#pragma unroll
        for (int m = 0; m < M; ++m) dr_store4(st, (m * 16 + l) * 4, dk, vec_state, S[m]);
    }
}

extern "C" int tl_delta_takes(int dk) { return dk > 0 && dk <= DR_MAX_DK ? 1 : 0; }

// q, k [T, >= (H / share) * dk], v [T, >= H * dv], b, a [T, >= H] float with row strides; rate_log [H], step_bias [H] or
// null; state: a request's [H, dv, dk] at state + slot * state_stride; out float [T, >= H * dv].  S sequences, rows
// q_start[s] .. q_start[s + 1].
extern "C" int tl_delta_walk(const float* q, int ldq, const float* k, int ldk, const float* v, int ldv, const float* b, int ldb,
                             const float* a, int lda, const float* rate_log, const float* step_bias, int share, float* state,
                             long long state_stride, const int32_t* state_slots, const int32_t* q_start, float* out, int ldo,
                             int S, int H, int dk, int dv, hipStream_t stream) {
    TL_CHECK_ARG(S >= 0 && H > 0 && dv > 0 && tl_delta_takes(dk), "tl_delta_walk: bad sizes S=%d H=%d dk=%d (at most %d) dv=%d", S, H, dk, DR_MAX_DK, dv);
    TL_CHECK_ARG(share >= 1 && H % share == 0, "tl_delta_walk: %d heads do not share queries and keys in groups of %d", H, share);
    TL_CHECK_ARG(ldq >= H / share * dk && ldk >= H / share * dk && ldv >= H * dv && ldo >= H * dv && ldb >= H && lda >= H, "tl_delta_walk: rows too short");
    TL_CHECK_ARG(rate_log && state_stride >= (long long)H * dk * dv, "tl_delta_walk: rates are missing or the state of a request is too small");
    TL_CHECK_ARG(H <= 65535 && S <= 65535, "tl_delta_walk: too many heads or sequences for one launch");
    if (S == 0) return 0;
    const int vec = ((uintptr_t)q % 16 == 0 && (uintptr_t)k % 16 == 0 && ldq % 4 == 0 && ldk % 4 == 0 && dk % 4 == 0) ? 1 : 0;
    const int vec_state = ((uintptr_t)state % 16 == 0 && state_stride % 4 == 0 && dk % 4 == 0) ? 1 : 0;
    dim3 grid(tl_ceil_div(dv, 16), H, S), block(DR_THREADS);
#define GO(M)                                                                                                                  \
    hipLaunchKernelGGL(delta_walk_kernel<M>, grid, block, 0, stream, q, ldq, k, ldk, v, ldv, b, ldb, a, lda, rate_log, step_bias, \
                       share, state, state_stride, state_slots, q_start, out, ldo, dk, dv, vec, vec_state)
    if (dk <= 64) GO(1);
    else if (dk <= 128) GO(2);
    else GO(4);
#undef GO
    TL_CHECK_LAUNCH("tl_delta_walk");
    return 0;
}

// ---- in chunks -----------------------------------------------------------------------------------------------
// four products with the k a lane's two 16-byte reads hold: row li of one operand and row li of the other at k = 4 lg .. + 3;
// the lane then holds D[4 lg + e][li]
__device__ __forceinline__ dr_f32x4 dr_mfma4(float4 a, float4 w, dr_f32x4 acc) {
    acc = __builtin_amdgcn_mfma_f32_16x16x4f32(a.x, w.x, acc, 0, 0, 0);
    acc = __builtin_amdgcn_mfma_f32_16x16x4f32(a.y, w.y, acc, 0, 0, 0);
    acc = __builtin_amdgcn_mfma_f32_16x16x4f32(a.z, w.z, acc, 0, 0, 0);
    acc = __builtin_amdgcn_mfma_f32_16x16x4f32(a.w, w.w, acc, 0, 0, 0);
    return acc;
}

// cs[t] = ln g_1 + .. + ln g_t for the chunk's n tokens (constant beyond), by the first wave, in both kernels that need it
__device__ __forceinline__ void dr_log_decays(const float* __restrict__ a, int lda, int t0, int n, int h, float rate, float bias,
                                              double* cs) {
    const int tid = threadIdx.x;
    if (tid < DR_L) {
        double run = tid < n ? (double)(-rate * dr_softplus(a[(size_t)(t0 + tid) * lda + h] + bias)) : 0.0;
#pragma unroll
        for (int off = 1; off < DR_L; off <<= 1) {           // inclusive sums over the lanes, in a fixed order
            const double below = __shfl_up(run, off, TL_WAVE);
            if (tid >= off) run += below;
        }
        cs[tid] = run;
    }
}

// A head's keys of the chunk into LDS rows of DP + 4 floats, zeros beyond the chunk's tokens and the head's dk.
template <int DP>
__device__ __forceinline__ void dr_fill_keys(const float* __restrict__ kh, int ldk, int t0, int n, int dk, int vec, float* Ks) {
    constexpr int PER = DR_L * DP / 4 / DR_THREADS;         // 1, 2, 4 or 8 pieces of four values per thread
    float4 r[PER];
#pragma unroll
    for (int u = 0; u < PER; ++u) {
        const int idx = threadIdx.x + u * DR_THREADS, tt = idx / (DP / 4), i = 4 * (idx % (DP / 4));
        r[u] = tt < n ? dr_load4(kh + (size_t)(t0 + tt) * ldk, i, dk, vec) : make_float4(0.f, 0.f, 0.f, 0.f);
    }
#pragma unroll
    for (int u = 0; u < PER; ++u) {
        const int idx = threadIdx.x + u * DR_THREADS, tt = idx / (DP / 4), i = 4 * (idx % (DP / 4));
        *reinterpret_cast<float4*>(&Ks[tt * (DP + 4) + i]) = r[u];
    }
}

// Per (head, chunk): U_0 [DR_L][dv], W [DR_L][DP], the decayed keys transposed [DP][DR_L] and exp(c_L).  The system is
// solved by forward substitution, a thread per column of the right-hand sides, its 64 unknowns in registers, a row of A
// read from LDS by all threads at once.
template <int DP>
__global__ __launch_bounds__(DR_THREADS) void delta_prepare_kernel(
    const float* __restrict__ k, int ldk, const float* __restrict__ v, int ldv, const float* __restrict__ b, int ldb,
    const float* __restrict__ a, int lda, const float* __restrict__ rate_log, const float* __restrict__ step_bias, int share,
    const int32_t* __restrict__ q_start, const int32_t* __restrict__ chunk_seq, const int32_t* __restrict__ chunk_row,
    float* __restrict__ ws_u0, float* __restrict__ ws_w, float* __restrict__ ws_kt, float* __restrict__ ws_dec, int H, int dk,
    int dv, int vec) {
    constexpr int LDK = DP + 4;
    extern __shared__ __attribute__((aligned(16))) float dr_smem[];
    float* Ks = dr_smem;                         // [DR_L][LDK]
    float* As = Ks + DR_L * LDK;                 // [DR_L][DR_LDA]: A, zeros on and above the diagonal
    double* cs = reinterpret_cast<double*>(As + DR_L * DR_LDA);   // [DR_L]
    float* bet = reinterpret_cast<float*>(cs + DR_L);             // [DR_L]
    const int h = blockIdx.x, c = blockIdx.y, tid = threadIdx.x;
    const int t0 = chunk_row[c], n = min(DR_L, q_start[chunk_seq[c] + 1] - t0);
    const size_t at = (size_t)c * H + h;
    dr_log_decays(a, lda, t0, n, h, expf(rate_log[h]), step_bias ? step_bias[h] : 0.f, cs);
    if (tid < DR_L) bet[tid] = tid < n ? dr_sigmoid(b[(size_t)(t0 + tid) * ldb + h]) : 0.f;
    dr_fill_keys<DP>(k + (size_t)(h / share) * dk, ldk, t0, n, dk, vec, Ks);
    __syncthreads();
    const int lane = tid & 63, wave = tid >> 6, li = lane & 15, lg = lane >> 4;
    {
        dr_f32x4 acc[DR_L / 16];
#pragma unroll
        for (int sb = 0; sb < DR_L / 16; ++sb) acc[sb] = dr_f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int kk = 0; kk < DP / 16; ++kk) {
            const float4 af = *reinterpret_cast<const float4*>(&Ks[(wave * 16 + li) * LDK + kk * 16 + 4 * lg]);
#pragma unroll
            for (int sb = 0; sb < DR_L / 16; ++sb)
                if (sb <= wave)
                    acc[sb] = dr_mfma4(af, *reinterpret_cast<const float4*>(&Ks[(sb * 16 + li) * LDK + kk * 16 + 4 * lg]), acc[sb]);
        }
#pragma unroll
        for (int sb = 0; sb < DR_L / 16; ++sb)
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                const int t = wave * 16 + 4 * lg + e, ss = sb * 16 + li;
                As[t * DR_LDA + ss] = ss < t ? bet[t] * expf((float)(cs[t] - cs[ss])) * acc[sb][e] : 0.f;
            }
    }
    // the decayed keys, transposed, and the chunk's whole decay
    const double c_end = cs[n - 1];
    for (int idx = tid; idx < DP * DR_L; idx += DR_THREADS) {
        const int i = idx >> 6, tt = idx & 63;
        ws_kt[at * (DP * DR_L) + idx] = tt < n ? expf((float)(c_end - cs[tt])) * Ks[tt * LDK + i] : 0.f;
    }
    if (tid == 0) ws_dec[at] = expf((float)c_end);
    __syncthreads();
    const int cols = dv + DP;
    for (int col = tid; col < cols; col += DR_THREADS) {
        float X[DR_L];
        if (col < dv) {
            const float* vc = v + (size_t)t0 * ldv + (size_t)h * dv + col;
#pragma unroll
            for (int t = 0; t < DR_L; ++t) X[t] = vc[(size_t)(t < n ? t : n - 1) * ldv];      // beyond the chunk beta is zero
#pragma unroll
            for (int t = 0; t < DR_L; ++t) X[t] *= bet[t];
        } else {
#pragma unroll
            for (int t = 0; t < DR_L; ++t) X[t] = bet[t] * expf((float)cs[t]) * Ks[t * LDK + col - dv];
        }
#pragma unroll
        for (int t = 1; t < DR_L; ++t) {
            float4 s = make_float4(0.f, 0.f, 0.f, 0.f);
#pragma unroll
            for (int m = 0; m < (t + 3) / 4; ++m) {           // entries on and above the diagonal are zero
                const float4 r = *reinterpret_cast<const float4*>(&As[t * DR_LDA + 4 * m]);
                s.x = __builtin_fmaf(r.x, X[4 * m], s.x);
                s.y = __builtin_fmaf(r.y, X[4 * m + 1], s.y);
                s.z = __builtin_fmaf(r.z, X[4 * m + 2], s.z);
                s.w = __builtin_fmaf(r.w, X[4 * m + 3], s.w);
            }
            X[t] -= (s.x + s.y) + (s.z + s.w);
        }
        float* dst = col < dv ? ws_u0 + at * (size_t)(DR_L * dv) + col : ws_w + at * (DR_L * DP) + (col - dv);
        const int ld = col < dv ? dv : DP;
#pragma unroll
        for (int t = 0; t < DR_L; ++t) dst[(size_t)t * ld] = X[t];
    }
}

// The chunks of a sequence in order, for one head and 16 value columns.  S lives in registers in the layout the matrix
// instruction leaves results in, wave w holding the blocks of 16 key rows w and w + 4, and goes through LDS (as does U) in
// the layout it reads operands in, which is the same: [block][lane group][lane] of four values.  The next chunk's operands
// are on their way in registers while a chunk is computed.
template <int NK>
__global__ __launch_bounds__(DR_THREADS) void delta_states_kernel(
    const float* __restrict__ ws_u0, const float* __restrict__ ws_w, const float* __restrict__ ws_kt,
    const float* __restrict__ ws_dec, float* __restrict__ ws_s, float* __restrict__ ws_ut, float* __restrict__ state,
    long long state_stride, const int32_t* __restrict__ state_slots, const int32_t* __restrict__ seq_chunk, int H, int dk, int dv) {
    constexpr int DP = NK * 16, NT = (NK + 3) / 4;
    __shared__ float4 Sl[NK * 64], Ul[4 * 64];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, li = lane & 15, lg = lane >> 4;
    const int j = blockIdx.x * 16 + li, h = blockIdx.y, s = blockIdx.z;
    const int c0 = seq_chunk[s], c1 = seq_chunk[s + 1];
    if (c1 <= c0) return;
    const bool col_ok = j < dv;
    float* st = state + (size_t)state_slots[s] * state_stride + ((size_t)h * dv + (col_ok ? j : 0)) * dk;
    dr_f32x4 S[NT];
#pragma unroll
    for (int m = 0; m < NT; ++m) {
        const int i = (wave + 4 * m) * 16 + 4 * lg;
#pragma unroll
        for (int e = 0; e < 4; ++e) S[m][e] = (col_ok && wave + 4 * m < NK && i + e < dk) ? st[i + e] : 0.f;
    }
    float4 wf[NK], kf[NT][4];
    float u0[4], dec;
    auto fetch = [&](int c, float4 (&W)[NK], float4 (&K)[NT][4], float (&U)[4], float& D) {
        const size_t at = (size_t)c * H + h;
        const float* w = ws_w + at * (DR_L * DP) + (wave * 16 + li) * DP + 4 * lg;
#pragma unroll
        for (int kk = 0; kk < NK; ++kk) W[kk] = *reinterpret_cast<const float4*>(w + 16 * kk);
#pragma unroll
        for (int m = 0; m < NT; ++m) {
            const int it = wave + 4 * m < NK ? wave + 4 * m : NK - 1;
            const float* kt = ws_kt + at * (DP * DR_L) + (it * 16 + li) * DR_L + 4 * lg;
#pragma unroll
            for (int kk = 0; kk < 4; ++kk) K[m][kk] = *reinterpret_cast<const float4*>(kt + 16 * kk);
        }
        const float* up = ws_u0 + at * (size_t)(DR_L * dv) + (size_t)(wave * 16 + 4 * lg) * dv + (col_ok ? j : 0);
#pragma unroll
        for (int e = 0; e < 4; ++e) U[e] = up[(size_t)e * dv];
        D = ws_dec[at];
    };
    fetch(c0, wf, kf, u0, dec);
    for (int c = c0; c < c1; ++c) {
        const size_t at = (size_t)c * H + h;
#pragma unroll
        for (int m = 0; m < NT; ++m) {
            const int it = wave + 4 * m;
            if (it < NK) {
                const float4 mine = make_float4(S[m][0], S[m][1], S[m][2], S[m][3]);
                Sl[(it * 4 + lg) * 16 + li] = mine;
                if (col_ok) *reinterpret_cast<float4*>(ws_s + at * (size_t)(dv * DP) + (size_t)j * DP + it * 16 + 4 * lg) = mine;
            }
        }
        __syncthreads();
        float4 wn[NK], kn[NT][4];
        float un[4], dn;
        fetch(c + 1 < c1 ? c + 1 : c, wn, kn, un, dn);
        dr_f32x4 p0 = dr_f32x4{0.f, 0.f, 0.f, 0.f}, p1 = p0;
#pragma unroll
        for (int kk = 0; kk < NK; ++kk) {
            if (kk & 1) p1 = dr_mfma4(wf[kk], Sl[(kk * 4 + lg) * 16 + li], p1);
            else p0 = dr_mfma4(wf[kk], Sl[(kk * 4 + lg) * 16 + li], p0);
        }
        const float4 U = make_float4(u0[0] - (p0[0] + p1[0]), u0[1] - (p0[1] + p1[1]), u0[2] - (p0[2] + p1[2]), u0[3] - (p0[3] + p1[3]));
        Ul[(wave * 4 + lg) * 16 + li] = U;
        if (col_ok) *reinterpret_cast<float4*>(ws_ut + at * (size_t)(dv * DR_L) + (size_t)j * DR_L + wave * 16 + 4 * lg) = U;
        __syncthreads();
#pragma unroll
        for (int m = 0; m < NT; ++m)
            if (wave + 4 * m < NK) {
                S[m] *= dec;
#pragma unroll
                for (int kk = 0; kk < 4; ++kk) S[m] = dr_mfma4(kf[m][kk], Ul[(kk * 4 + lg) * 16 + li], S[m]);
            }
#pragma unroll
        for (int kk = 0; kk < NK; ++kk) wf[kk] = wn[kk];
#pragma unroll
        for (int m = 0; m < NT; ++m)
#pragma unroll
            for (int kk = 0; kk < 4; ++kk) kf[m][kk] = kn[m][kk];
#pragma unroll
        for (int e = 0; e < 4; ++e) u0[e] = un[e];
        dec = dn;
    }
#pragma unroll
    for (int m = 0; m < NT; ++m) {
        const int i = (wave + 4 * m) * 16 + 4 * lg;
#pragma unroll
        for (int e = 0; e < 4; ++e)
            if (col_ok && wave + 4 * m < NK && i + e < dk) st[i + e] = S[m][e];
    }
}

// Per (head, chunk): wave w owns tokens 16 w .. 16 w + 15.  The chunk's matrix exp(c_t - c_s) (q_t . k_s), s <= t, goes
// through LDS within the wave; the entering state and U are read in operand layout straight from the workspace.
template <int NK>
__global__ __launch_bounds__(DR_THREADS) void delta_outputs_kernel(
    const float* __restrict__ q, int ldq, const float* __restrict__ k, int ldk, const float* __restrict__ a, int lda,
    const float* __restrict__ rate_log, const float* __restrict__ step_bias, int share, const int32_t* __restrict__ q_start,
    const int32_t* __restrict__ chunk_seq, const int32_t* __restrict__ chunk_row, const float* __restrict__ ws_s,
    const float* __restrict__ ws_ut, float* __restrict__ out, int ldo, int H, int dk, int dv, int vec) {
    constexpr int DP = NK * 16, LDK = DP + 4;
    extern __shared__ __attribute__((aligned(16))) float dr_smem[];
    float* Ks = dr_smem;                         // [DR_L][LDK]
    float* Ms = Ks + DR_L * LDK;                 // [DR_L][DR_LDA]
    double* cs = reinterpret_cast<double*>(Ms + DR_L * DR_LDA);
    const int h = blockIdx.x, c = blockIdx.y, tid = threadIdx.x;
    const int t0 = chunk_row[c], n = min(DR_L, q_start[chunk_seq[c] + 1] - t0);
    const size_t at = (size_t)c * H + h;
    const int lane = tid & 63, wave = tid >> 6, li = lane & 15, lg = lane >> 4;
    float4 qf[NK];
    {
        const int tt = wave * 16 + li;
        const float* qr = q + (size_t)(t0 + (tt < n ? tt : 0)) * ldq + (size_t)(h / share) * dk;
#pragma unroll
        for (int kk = 0; kk < NK; ++kk)
            qf[kk] = tt < n ? dr_load4(qr, 16 * kk + 4 * lg, dk, vec) : make_float4(0.f, 0.f, 0.f, 0.f);
    }
    dr_log_decays(a, lda, t0, n, h, expf(rate_log[h]), step_bias ? step_bias[h] : 0.f, cs);
    dr_fill_keys<DP>(k + (size_t)(h / share) * dk, ldk, t0, n, dk, vec, Ks);
    __syncthreads();
    if (wave * 16 >= n) return;                  // no barrier follows
    {
        dr_f32x4 acc[DR_L / 16];
#pragma unroll
        for (int sb = 0; sb < DR_L / 16; ++sb) acc[sb] = dr_f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int kk = 0; kk < NK; ++kk) {
#pragma unroll
            for (int sb = 0; sb < DR_L / 16; ++sb)
                if (sb <= wave)
                    acc[sb] = dr_mfma4(qf[kk], *reinterpret_cast<const float4*>(&Ks[(sb * 16 + li) * LDK + kk * 16 + 4 * lg]), acc[sb]);
        }
#pragma unroll
        for (int sb = 0; sb < DR_L / 16; ++sb)
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                const int t = wave * 16 + 4 * lg + e, ss = sb * 16 + li;
                Ms[t * DR_LDA + ss] = ss <= t ? acc[sb][e] * expf((float)(cs[t] - cs[ss])) : 0.f;
            }
    }
    // Ms rows of this wave are written and read by this wave only; LDS operations of a wave complete in order
    __builtin_amdgcn_fence(__ATOMIC_RELEASE, "wavefront");
    __builtin_amdgcn_wave_barrier();
    __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "wavefront");
    float4 mf[DR_L / 16];
#pragma unroll
    for (int sb = 0; sb < DR_L / 16; ++sb) mf[sb] = *reinterpret_cast<const float4*>(&Ms[(wave * 16 + li) * DR_LDA + sb * 16 + 4 * lg]);
    const float into = expf((float)cs[wave * 16 + li]);      // the factor on the entering state, for this lane's row
#pragma unroll
    for (int kk = 0; kk < NK; ++kk) qf[kk].x *= into, qf[kk].y *= into, qf[kk].z *= into, qf[kk].w *= into;
    const float* S0 = ws_s + at * (size_t)(dv * DP);          // [dv][DP]
    const float* UT = ws_ut + at * (size_t)(dv * DR_L);       // [dv][DR_L]
    for (int j0 = 0; j0 < dv; j0 += 32) {
        float4 sf[2][NK], uf[2][DR_L / 16];
#pragma unroll
        for (int x = 0; x < 2; ++x) {
            const int j = j0 + 16 * x + li, jc = j < dv ? j : dv - 1;
#pragma unroll
            for (int kk = 0; kk < NK; ++kk) sf[x][kk] = *reinterpret_cast<const float4*>(S0 + (size_t)jc * DP + 16 * kk + 4 * lg);
#pragma unroll
            for (int sb = 0; sb < DR_L / 16; ++sb)
                if (sb <= wave) uf[x][sb] = *reinterpret_cast<const float4*>(UT + (size_t)jc * DR_L + 16 * sb + 4 * lg);
        }
        dr_f32x4 y[2];
        y[0] = y[1] = dr_f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int kk = 0; kk < NK; ++kk)
#pragma unroll
            for (int x = 0; x < 2; ++x) y[x] = dr_mfma4(qf[kk], sf[x][kk], y[x]);
#pragma unroll
        for (int sb = 0; sb < DR_L / 16; ++sb)
            if (sb <= wave) {
#pragma unroll
                for (int x = 0; x < 2; ++x) y[x] = dr_mfma4(mf[sb], uf[x][sb], y[x]);
            }
#pragma unroll
        for (int x = 0; x < 2; ++x) {
            const int j = j0 + 16 * x + li;
            if (j >= dv) continue;
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                const int t = wave * 16 + 4 * lg + e;
                if (t < n) out[(size_t)(t0 + t) * ldo + (size_t)h * dv + j] = y[x][e];
            }
        }
    }
}

static int dr_padded_keys(int dk) { return dk <= 16 ? 16 : dk <= 32 ? 32 : dk <= 64 ? 64 : 128; }

extern "C" int tl_delta_chunked_takes(int dk, int dv) { return dk > 0 && dk <= 128 && dv > 0 ? 1 : 0; }
extern "C" int tl_delta_chunk_tokens() { return DR_L; }
// floats of workspace per chunk and head
extern "C" long long tl_delta_chunked_workspace(int dk, int dv) {
    const long long DP = dr_padded_keys(dk);
    return 2LL * DR_L * dv + 2LL * DR_L * DP + (long long)dv * DP + 4;
}

// The operands of tl_delta_walk.  chunk_seq, chunk_row [NC]: a chunk's sequence and its first row of the step (a sequence's
// rows in chunks of DR_L from its first row on); seq_chunk [S + 1]: a sequence's first chunk.  ws: NC * H *
// tl_delta_chunked_workspace floats, 16-byte aligned.
extern "C" int tl_delta_chunked(const float* q, int ldq, const float* k, int ldk, const float* v, int ldv, const float* b, int ldb,
                                const float* a, int lda, const float* rate_log, const float* step_bias, int share, float* state,
                                long long state_stride, const int32_t* state_slots, const int32_t* q_start,
                                const int32_t* chunk_seq, const int32_t* chunk_row, const int32_t* seq_chunk, float* ws, float* out,
                                int ldo, int S, int NC, int H, int dk, int dv, hipStream_t stream) {
    TL_CHECK_ARG(S >= 0 && NC >= 0 && H > 0 && tl_delta_chunked_takes(dk, dv), "tl_delta_chunked: bad sizes S=%d H=%d dk=%d dv=%d", S, H, dk, dv);
    TL_CHECK_ARG(share >= 1 && H % share == 0, "tl_delta_chunked: %d heads do not share queries and keys in groups of %d", H, share);
    TL_CHECK_ARG(ldq >= H / share * dk && ldk >= H / share * dk && ldv >= H * dv && ldo >= H * dv && ldb >= H && lda >= H, "tl_delta_chunked: rows too short");
    TL_CHECK_ARG(rate_log && state_stride >= (long long)H * dk * dv, "tl_delta_chunked: rates are missing or the state of a request is too small");
    TL_CHECK_ARG(NC <= 65535 && H <= 65535 && S <= 65535, "tl_delta_chunked: too many chunks, heads or sequences for one launch");
    if (S == 0 || NC == 0) return 0;
    TL_CHECK_ARG(ws && (uintptr_t)ws % 16 == 0 && chunk_seq && chunk_row && seq_chunk, "tl_delta_chunked: the workspace (16-byte aligned) or the chunk tables are missing");
    const int vec = ((uintptr_t)q % 16 == 0 && (uintptr_t)k % 16 == 0 && ldq % 4 == 0 && ldk % 4 == 0 && dk % 4 == 0) ? 1 : 0;
    const int DP = dr_padded_keys(dk);
    const size_t nh = (size_t)NC * H;
    float* ws_w = ws;                            // pieces that are read in 16-byte units first
    float* ws_kt = ws_w + nh * DR_L * DP;
    float* ws_s = ws_kt + nh * DR_L * DP;
    float* ws_ut = ws_s + nh * dv * DP;
    float* ws_u0 = ws_ut + nh * dv * DR_L;
    float* ws_dec = ws_u0 + nh * dv * DR_L;
    const size_t lds = sizeof(float) * (DR_L * (DP + 4) + DR_L * DR_LDA + DR_L) + sizeof(double) * DR_L;
#define GO(NK)                                                                                                                   \
    do {                                                                                                                         \
        hipLaunchKernelGGL(delta_prepare_kernel<16 * NK>, dim3(H, NC), dim3(DR_THREADS), lds, stream, k, ldk, v, ldv, b, ldb, a, lda, \
                           rate_log, step_bias, share, q_start, chunk_seq, chunk_row, ws_u0, ws_w, ws_kt, ws_dec, H, dk, dv, vec); \
        TL_CHECK_LAUNCH("tl_delta_chunked prepare");                                                                             \
        hipLaunchKernelGGL(delta_states_kernel<NK>, dim3(tl_ceil_div(dv, 16), H, S), dim3(DR_THREADS), 0, stream, ws_u0, ws_w, ws_kt, \
                           ws_dec, ws_s, ws_ut, state, state_stride, state_slots, seq_chunk, H, dk, dv);                          \
        TL_CHECK_LAUNCH("tl_delta_chunked states");                                                                              \
        hipLaunchKernelGGL(delta_outputs_kernel<NK>, dim3(H, NC), dim3(DR_THREADS), lds, stream, q, ldq, k, ldk, a, lda, rate_log,  \
                           step_bias, share, q_start, chunk_seq, chunk_row, ws_s, ws_ut, out, ldo, H, dk, dv, vec);               \
        TL_CHECK_LAUNCH("tl_delta_chunked outputs");                                                                             \
    } while (0)
    if (DP == 16) GO(1);
    else if (DP == 32) GO(2);
    else if (DP == 64) GO(4);
    else GO(8);
#undef GO
    return 0;
}
