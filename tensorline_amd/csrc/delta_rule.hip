// The gated delta rule over a matrix state per head, kept per request between steps:
//
//     u_t = beta_t (v_t - g_t S_(t-1)^T k_t),   S_t = g_t S_(t-1) + k_t u_t^T,   o_t = S_t^T q_t
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
//          diag(beta exp c) K, and forms what else a chunk needs of its keys and queries, all chunks at once;
//       2. delta_states_kernel walks the chunks of a sequence, a work-group per head and 16 value columns: U = U_0 - W S_0,
//          o_t = exp(c_t) S_0^T q_t + sum_(s <= t) exp(c_t - c_s) (q_t . k_s) u_s, S_L = exp(c_L) S_0 + sum_s exp(c_L - c_s) k_s u_s^T.
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
    int dv, int vec, int vec_state, int upto) {
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, l = lane & 15;
    const int j = blockIdx.x * 16 + wave * 4 + (lane >> 4), h = blockIdx.y, s = blockIdx.z;
    const int r0 = q_start[s], r1 = q_start[s + 1];
    if (r1 <= r0 || r1 - r0 > upto) return;
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
// q_start[s] .. q_start[s + 1]; upto > 0: only the sequences that bring at most so many rows are walked.
extern "C" int tl_delta_walk(const float* q, int ldq, const float* k, int ldk, const float* v, int ldv, const float* b, int ldb,
                             const float* a, int lda, const float* rate_log, const float* step_bias, int share, float* state,
                             long long state_stride, const int32_t* state_slots, const int32_t* q_start, float* out, int ldo,
                             int S, int H, int dk, int dv, int upto, hipStream_t stream) {
    if (upto <= 0) upto = 0x7fffffff;
    TL_CHECK_ARG(S >= 0 && H > 0 && dv > 0 && tl_delta_takes(dk),
                 "tl_delta_walk: bad sizes S=%d H=%d dk=%d (at most %d) dv=%d", S, H, dk, DR_MAX_DK, dv);
    TL_CHECK_ARG(share >= 1 && H % share == 0, "tl_delta_walk: %d heads do not share queries and keys in groups of %d", H, share);
    TL_CHECK_ARG(ldq >= H / share * dk && ldk >= H / share * dk && ldv >= H * dv && ldo >= H * dv && ldb >= H && lda >= H,
                 "tl_delta_walk: rows too short");
    TL_CHECK_ARG(rate_log && state_stride >= (long long)H * dk * dv,
                 "tl_delta_walk: rates are missing or the state of a request is too small");
    TL_CHECK_ARG(H <= 65535 && S <= 65535, "tl_delta_walk: too many heads or sequences for one launch");
    if (S == 0) return 0;
    const int vec = ((uintptr_t)q % 16 == 0 && (uintptr_t)k % 16 == 0 && ldq % 4 == 0 && ldk % 4 == 0 && dk % 4 == 0) ? 1 : 0;
    const int vec_state = ((uintptr_t)state % 16 == 0 && state_stride % 4 == 0 && dk % 4 == 0) ? 1 : 0;
    dim3 grid(tl_ceil_div(dv, 16), H, S), block(DR_THREADS);
#define GO(M)                                                                                                                  \
    hipLaunchKernelGGL(delta_walk_kernel<M>, grid, block, 0, stream, q, ldq, k, ldk, v, ldv, b, ldb, a, lda, rate_log, step_bias, \
                       share, state, state_stride, state_slots, q_start, out, ldo, dk, dv, vec, vec_state, upto)
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

// one of those four products; independent ones are issued in turn (a dependent one waits half as long again)
template <int E>
__device__ __forceinline__ dr_f32x4 dr_mfma1(float4 a, float4 w, dr_f32x4 acc) {
    return __builtin_amdgcn_mfma_f32_16x16x4f32(E == 0 ? a.x : E == 1 ? a.y : E == 2 ? a.z : a.w,
                                                E == 0 ? w.x : E == 1 ? w.y : E == 2 ? w.z : w.w, acc, 0, 0, 0);
}
template <bool V>
struct DrFlag {
    static constexpr bool value = V;
};
#define DR_EACH4(STEP) STEP(0) STEP(1) STEP(2) STEP(3)
__device__ __forceinline__ float4 dr_f4(dr_f32x4 v) { return make_float4(v[0], v[1], v[2], v[3]); }

// cs[t] = ln g_1 + .. + ln g_t for the chunk's n tokens (constant beyond), by the first wave
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

// A head's queries or keys of the chunk: from memory into registers, zeros beyond the chunk's tokens and the head's dk, and
// from there into LDS rows of DP + 4 floats.
template <int DP>
struct DrTile {
    static constexpr int PER = DR_L * DP / 4 / DR_THREADS;   // 1, 2, 4 or 8 pieces of four values per thread
    float4 r[PER];
    __device__ __forceinline__ void load(const float* __restrict__ src, int ld, int t0, int n, int dk, int vec) {
#pragma unroll
        for (int u = 0; u < PER; ++u) {
            const int idx = threadIdx.x + u * DR_THREADS, tt = idx / (DP / 4), i = 4 * (idx % (DP / 4));
            r[u] = tt < n ? dr_load4(src + (size_t)(t0 + tt) * ld, i, dk, vec) : make_float4(0.f, 0.f, 0.f, 0.f);
        }
    }
    __device__ __forceinline__ void stash(float* rows) const {
#pragma unroll
        for (int u = 0; u < PER; ++u) {
            const int idx = threadIdx.x + u * DR_THREADS, tt = idx / (DP / 4), i = 4 * (idx % (DP / 4));
            *reinterpret_cast<float4*>(&rows[tt * (DP + 4) + i]) = r[u];
        }
    }
};

// Per (head, chunk): U_0, W, the decayed keys transposed, the queries times exp(c_t), the outputs' matrix M_ts = exp(c_t - c_s)
// (q_t . k_s), s <= t, and exp(c_L); each as the next kernel's operands, in blocks of 16 x 16 laid out [lane][4] as a lane
// reads them, so that a block is one kilobyte in a row.  (Read row by row, a wave's load of an operand touches sixteen rows
// in every quarter of it, which takes four times as long.)  The system is solved in blocks of 16 tokens: the diagonal
// blocks I + A_ii are inverted by substitution (a lane per column), then X_i = (I + A_ii)^-1 (R_i - sum_(j < i) A_ij X_j)
// runs on the matrix instruction, 16 columns of a right-hand side at a time: what it leaves in a lane is in the layout it
// reads its second operand in, so solved blocks are used as they are; with its operands exchanged the instruction leaves
// the transposed block, which is the layout of a first operand, as W is needed.
template <int DP>
__global__ __launch_bounds__(DR_THREADS) void delta_prepare_kernel(
    const float* __restrict__ q, int ldq, const float* __restrict__ k, int ldk, const float* __restrict__ v, int ldv,
    const float* __restrict__ b, int ldb, const float* __restrict__ a, int lda, const float* __restrict__ rate_log,
    const float* __restrict__ step_bias, int share, const int32_t* __restrict__ q_start, const int32_t* __restrict__ chunk_seq,
    const int32_t* __restrict__ chunk_row, float* __restrict__ ws_u0, float* __restrict__ ws_w, float* __restrict__ ws_kt,
    float* __restrict__ ws_m, float* __restrict__ ws_q, float* __restrict__ ws_dec, int H, int dk, int dv, int vec) {
    constexpr int LDK = DP + 4, NB = DR_L / 16, LDI = 20;
    __shared__ __attribute__((aligned(16))) float Ks[DR_L * LDK];
    __shared__ __attribute__((aligned(16))) float As[DR_L * DR_LDA];      // zeros on and above the diagonal
    __shared__ __attribute__((aligned(16))) float Ti[NB * 16 * LDI];      // the inverted diagonal blocks
    __shared__ double cs[DR_L];
    __shared__ float bet[DR_L], bin[DR_L], into[DR_L];                    // beta_t, beta_t exp(c_t) (zero beyond the chunk), exp(c_t)
    const int h = blockIdx.x, c = blockIdx.y, tid = threadIdx.x;
    const int t0 = chunk_row[c], n = min(DR_L, q_start[chunk_seq[c] + 1] - t0);
    const size_t at = (size_t)c * H + h;
    const int lane = tid & 63, wave = tid >> 6, li = lane & 15, lg = lane >> 4;
    DrTile<DP> qt, kt;
    qt.load(q + (size_t)(h / share) * dk, ldq, t0, n, dk, vec);
    kt.load(k + (size_t)(h / share) * dk, ldk, t0, n, dk, vec);
    // the values of this wave's first pair of column blocks are on their way from here on
    const int vt = (dv + 15) >> 4;
    dr_f32x4 V[2][NB];
    auto load_values = [&](int ct) {
#pragma unroll
        for (int x = 0; x < 2; ++x) {
            const int j = (ct + 4 * x) * 16 + li;
            const float* vc = v + (size_t)t0 * ldv + (size_t)h * dv + (j < dv ? j : dv - 1);
#pragma unroll
            for (int i = 0; i < NB; ++i)
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    const int t = 16 * i + 4 * lg + e;
                    V[x][i][e] = vc[(size_t)(t < n ? t : n - 1) * ldv];    // beyond the chunk beta is zero
                }
        }
    };
    load_values(wave);
    dr_log_decays(a, lda, t0, n, h, expf(rate_log[h]), step_bias ? step_bias[h] : 0.f, cs);
    if (tid < DR_L) {
        const float beta = tid < n ? dr_sigmoid(b[(size_t)(t0 + tid) * ldb + h]) : 0.f;
        const float in = expf((float)cs[tid]);
        bet[tid] = beta;
        bin[tid] = beta * in;
        into[tid] = in;
    }
    // the queries pass through the keys' place
    qt.stash(Ks);
    __syncthreads();
    float4 qf[DP / 16];
#pragma unroll
    for (int kk = 0; kk < DP / 16; ++kk) qf[kk] = *reinterpret_cast<const float4*>(&Ks[(wave * 16 + li) * LDK + kk * 16 + 4 * lg]);
    {
        const float in = into[wave * 16 + li];
        float4* dst = reinterpret_cast<float4*>(ws_q + at * (DR_L * DP)) + wave * (DP / 16) * 64 + lane;
#pragma unroll
        for (int kk = 0; kk < DP / 16; ++kk) dst[kk * 64] = make_float4(qf[kk].x * in, qf[kk].y * in, qf[kk].z * in, qf[kk].w * in);
    }
    __syncthreads();
    kt.stash(Ks);
    __syncthreads();
    {
        dr_f32x4 ka[NB], qa[NB];
#pragma unroll
        for (int sb = 0; sb < NB; ++sb) ka[sb] = qa[sb] = dr_f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int kk = 0; kk < DP / 16; ++kk) {
            const float4 kf = *reinterpret_cast<const float4*>(&Ks[(wave * 16 + li) * LDK + kk * 16 + 4 * lg]);
#pragma unroll
            for (int sb = 0; sb < NB; ++sb)
                if (sb <= wave) {
                    const float4 other = *reinterpret_cast<const float4*>(&Ks[(sb * 16 + li) * LDK + kk * 16 + 4 * lg]);
#define DR_STEP(E)                                   \
    ka[sb] = dr_mfma1<E>(kf, other, ka[sb]);         \
    qa[sb] = dr_mfma1<E>(other, qf[kk], qa[sb]);     /* transposed */
                    DR_EACH4(DR_STEP)
#undef DR_STEP
                }
        }
        float4* M = reinterpret_cast<float4*>(ws_m + at * (DR_L * DR_L)) + wave * NB * 64 + lane;
#pragma unroll
        for (int sb = 0; sb < NB; ++sb) {
            float m[4];
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                const int t = wave * 16 + 4 * lg + e, ss = sb * 16 + li;                  // this lane of K K^T
                As[t * DR_LDA + ss] = ss < t ? bet[t] * expf((float)(cs[t] - cs[ss])) * ka[sb][e] : 0.f;
                const int tq = wave * 16 + li, sq = sb * 16 + 4 * lg + e;                 // this lane of (Q K^T)^T
                m[e] = sq <= tq ? expf((float)(cs[tq] - cs[sq])) * qa[sb][e] : 0.f;
            }
            if (sb <= wave) M[sb * 64] = make_float4(m[0], m[1], m[2], m[3]);
        }
    }
    // the decayed keys, transposed, and the chunk's whole decay
    const double c_end = cs[n - 1];
    {
        float out_of[NB][4];
#pragma unroll
        for (int kk = 0; kk < NB; ++kk)
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                const int tt = 16 * kk + 4 * lg + e;
                out_of[kk][e] = tt < n ? expf((float)(c_end - cs[tt])) : 0.f;
            }
        float4* dst = reinterpret_cast<float4*>(ws_kt + at * (DP * DR_L)) + lane;
        for (int it = wave; it < DP / 16; it += DR_THREADS / 64)
#pragma unroll
            for (int kk = 0; kk < NB; ++kk) {
                const float* col = &Ks[(16 * kk + 4 * lg) * LDK + it * 16 + li];
                dst[(it * NB + kk) * 64] = make_float4(out_of[kk][0] * col[0], out_of[kk][1] * col[LDK], out_of[kk][2] * col[2 * LDK],
                                                       out_of[kk][3] * col[3 * LDK]);
            }
    }
    if (tid == 0) ws_dec[at] = expf((float)c_end);
    __syncthreads();
    {
        float x[16];
#pragma unroll
        for (int i = 0; i < 16; ++i) {
            float sum = 0.f;
#pragma unroll
            for (int m4 = 0; m4 < (i + 3) / 4; ++m4) {
                const float4 r = *reinterpret_cast<const float4*>(&As[(wave * 16 + i) * DR_LDA + wave * 16 + 4 * m4]);
                sum = __builtin_fmaf(r.x, x[4 * m4], sum);
                if (4 * m4 + 1 < i) sum = __builtin_fmaf(r.y, x[4 * m4 + 1], sum);
                if (4 * m4 + 2 < i) sum = __builtin_fmaf(r.z, x[4 * m4 + 2], sum);
                if (4 * m4 + 3 < i) sum = __builtin_fmaf(r.w, x[4 * m4 + 3], sum);
            }
            x[i] = (i == li ? 1.0f : 0.f) - sum;
            if (lg == 0) Ti[(wave * 16 + i) * LDI + li] = x[i];
        }
    }
    __syncthreads();
    float4 af[NB][NB];                                                     // A_ij below the diagonal, the inverses on it
#pragma unroll
    for (int i = 0; i < NB; ++i)
#pragma unroll
        for (int j = 0; j <= i; ++j)
            af[i][j] = j < i ? *reinterpret_cast<const float4*>(&As[(i * 16 + li) * DR_LDA + j * 16 + 4 * lg])
                             : *reinterpret_cast<const float4*>(&Ti[(i * 16 + li) * LDI + 4 * lg]);
    // a pair of blocks of 16 columns at a time: their chains of dependent products are issued in turn
    auto solve = [&](dr_f32x4 (&X)[2][NB], auto transposed, dr_f32x4 (&Y)[2][NB]) {
#pragma unroll
        for (int i = 0; i < NB; ++i) {
            dr_f32x4 a0 = dr_f32x4{0.f, 0.f, 0.f, 0.f}, a1 = a0;
#pragma unroll
            for (int j = 0; j < i; ++j) {
                const float4 x0 = dr_f4(X[0][j]), x1 = dr_f4(X[1][j]);
#define DR_STEP(E)                              \
    a0 = dr_mfma1<E>(af[i][j], x0, a0);         \
    a1 = dr_mfma1<E>(af[i][j], x1, a1);
                DR_EACH4(DR_STEP)
#undef DR_STEP
            }
            const float4 r0 = dr_f4(X[0][i] - a0), r1 = dr_f4(X[1][i] - a1);
            a0 = a1 = dr_f32x4{0.f, 0.f, 0.f, 0.f};
#define DR_STEP(E)                              \
    a0 = dr_mfma1<E>(af[i][i], r0, a0);         \
    a1 = dr_mfma1<E>(af[i][i], r1, a1);
            DR_EACH4(DR_STEP)
#undef DR_STEP
            X[0][i] = a0;
            X[1][i] = a1;
            if (transposed.value) {
                a0 = a1 = dr_f32x4{0.f, 0.f, 0.f, 0.f};
#define DR_STEP(E)                              \
    a0 = dr_mfma1<E>(r0, af[i][i], a0);         \
    a1 = dr_mfma1<E>(r1, af[i][i], a1);
                DR_EACH4(DR_STEP)
#undef DR_STEP
                Y[0][i] = a0;
                Y[1][i] = a1;
            }
        }
    };
    dr_f32x4 Y[2][NB];
    float4* u0 = reinterpret_cast<float4*>(ws_u0 + at * (size_t)(vt * 16 * DR_L)) + lane;
    for (int ct = wave; ct < vt; ct += 8) {
        if (ct != wave) load_values(ct);
#pragma unroll
        for (int x = 0; x < 2; ++x)
#pragma unroll
            for (int i = 0; i < NB; ++i)
#pragma unroll
                for (int e = 0; e < 4; ++e) V[x][i][e] *= bet[16 * i + 4 * lg + e];
        solve(V, DrFlag<false>{}, Y);
#pragma unroll
        for (int x = 0; x < 2; ++x)
            if (ct + 4 * x < vt) {
#pragma unroll
                for (int i = 0; i < NB; ++i) u0[((ct + 4 * x) * NB + i) * 64] = dr_f4(V[x][i]);
            }
    }
    for (int ct = wave; ct < DP / 16; ct += 8) {
#pragma unroll
        for (int x = 0; x < 2; ++x) {
            const int col = ((ct + 4 * x < DP / 16 ? ct + 4 * x : ct) << 4) + li;
#pragma unroll
            for (int i = 0; i < NB; ++i)
#pragma unroll
                for (int e = 0; e < 4; ++e) V[x][i][e] = bin[16 * i + 4 * lg + e] * Ks[(16 * i + 4 * lg + e) * LDK + col];
        }
        solve(V, DrFlag<true>{}, Y);
        float4* dst = reinterpret_cast<float4*>(ws_w + at * (DR_L * DP)) + lane;
#pragma unroll
        for (int x = 0; x < 2; ++x)
            if (ct + 4 * x < DP / 16) {
#pragma unroll
                for (int i = 0; i < NB; ++i) dst[(i * (DP / 16) + ct + 4 * x) * 64] = dr_f4(Y[x][i]);
            }
    }
}

// The chunks of a sequence in order, for one head and 16 value columns: U = U_0 - W S, the outputs S^T (exp(c_t) q_t) + M U, S <-
// exp(c_L) S + (decayed keys)^T U.  S lives in registers in the layout the matrix instruction leaves results in, wave w
// holding the blocks of 16 key rows w and w + 4, and goes through LDS (as does U) in the layout it reads operands in, which
// is the same: [block][lane group][lane] of four values.  Wave w has tokens 16 w .. 16 w + 15 of U and of the outputs.  A
// step's operands are asked for as soon as the step before has used its own, into the same registers.
template <int NK>
__global__ __launch_bounds__(DR_THREADS) __attribute__((amdgpu_waves_per_eu(1, 1))) void delta_states_kernel(
    const float* __restrict__ ws_u0, const float* __restrict__ ws_w, const float* __restrict__ ws_kt,
    const float* __restrict__ ws_m, const float* __restrict__ ws_q, const float* __restrict__ ws_dec,
    float* __restrict__ state, long long state_stride,
    const int32_t* __restrict__ state_slots, const int32_t* __restrict__ q_start, const int32_t* __restrict__ seq_chunk,
    float* __restrict__ out, int ldo, int H, int dk, int dv) {
    constexpr int DP = NK * 16, NT = (NK + 3) / 4;
    __shared__ float4 Sl[NK * 64], Ul[4 * 64];
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), li = lane & 15, lg = lane >> 4;
    // heads vary fastest: with heads a multiple of 8, the column blocks of a head, which read the same W, keys and M, lie on one
    // XCD and share its L2
    const int j = blockIdx.y * 16 + li, h = blockIdx.x, s = blockIdx.z;
    const int c0 = seq_chunk[s], c1 = seq_chunk[s + 1];
    if (c1 <= c0) return;
    const int row0 = q_start[s], row1 = q_start[s + 1], vt = (dv + 15) >> 4;
    const bool col_ok = j < dv;
    float* st = state + (size_t)state_slots[s] * state_stride + ((size_t)h * dv + (col_ok ? j : 0)) * dk;
    dr_f32x4 S[NT];
#pragma unroll
    for (int m = 0; m < NT; ++m) {
        const int i = (wave + 4 * m) * 16 + 4 * lg;
#pragma unroll
        for (int e = 0; e < 4; ++e) S[m][e] = (col_ok && wave + 4 * m < NK && i + e < dk) ? st[i + e] : 0.f;
    }
    float4 wf[NK], qf[NK], kf[NT][4], mf[4], u0;
    float dec;
    auto fetch_wq = [&](int c) {
        const size_t at = (size_t)c * H + h;
        const float4* w = reinterpret_cast<const float4*>(ws_w + at * (DR_L * DP)) + wave * NK * 64 + lane;
        const float4* qs = reinterpret_cast<const float4*>(ws_q + at * (DR_L * DP)) + wave * NK * 64 + lane;
#pragma unroll
        for (int kk = 0; kk < NK; ++kk) {
            wf[kk] = w[kk * 64];
            qf[kk] = qs[kk * 64];
        }
    };
    auto fetch_u = [&](int c) {
        const size_t at = (size_t)c * H + h;
        u0 = reinterpret_cast<const float4*>(ws_u0 + at * (size_t)(vt * 16 * DR_L))[((size_t)blockIdx.y * 4 + wave) * 64 + lane];
        dec = ws_dec[at];
    };
    auto fetch_k = [&](int c) {
        const size_t at = (size_t)c * H + h;
        const float4* kt = reinterpret_cast<const float4*>(ws_kt + at * (DP * DR_L)) + lane;
#pragma unroll
        for (int kk = 0; kk < 4; ++kk)
#pragma unroll
            for (int m = 0; m < NT; ++m) kf[m][kk] = kt[((wave + 4 * m < NK ? wave + 4 * m : NK - 1) * 4 + kk) * 64];
        const float4* mm = reinterpret_cast<const float4*>(ws_m + at * (DR_L * DR_L)) + wave * 4 * 64 + lane;
#pragma unroll
        for (int kk = 0; kk < 4; ++kk)                       // blocks above the diagonal are not kept
            mf[kk] = kk <= wave ? mm[kk * 64] : make_float4(0.f, 0.f, 0.f, 0.f);
    };
    // In the order in which a step uses them, here as in the loop: a wait for the first ones is then no wait for the last.
    fetch_wq(c0);
    __builtin_amdgcn_sched_barrier(0);
    fetch_u(c0);
    __builtin_amdgcn_sched_barrier(0);
    fetch_k(c0);
    __builtin_amdgcn_sched_barrier(0);
    for (int c = c0; c < c1; ++c) {
        const int cn = c + 1 < c1 ? c + 1 : c;
#pragma unroll
        for (int m = 0; m < NT; ++m)
            if (wave + 4 * m < NK) Sl[((wave + 4 * m) * 4 + lg) * 16 + li] = make_float4(S[m][0], S[m][1], S[m][2], S[m][3]);
        __syncthreads();
        float4 sf[NK];
#pragma unroll
        for (int kk = 0; kk < NK; ++kk) sf[kk] = Sl[(kk * 4 + lg) * 16 + li];
        __builtin_amdgcn_sched_barrier(0);           // all of it asked for before the first product waits
        // two chains of dependent products in turn, U's first: the others hide the wait for it
        const dr_f32x4 zero = dr_f32x4{0.f, 0.f, 0.f, 0.f};
        dr_f32x4 p0 = zero, p1 = zero, y0 = zero, y1 = zero;
#pragma unroll
        for (int kk = 0; kk < NK; kk += 2) {
#define DR_STEP(E)                                           \
    p0 = dr_mfma1<E>(wf[kk], sf[kk], p0);                    \
    if (kk + 1 < NK) p1 = dr_mfma1<E>(wf[kk + 1], sf[kk + 1], p1);
            DR_EACH4(DR_STEP)
#undef DR_STEP
        }
        p0 += p1;
        Ul[(wave * 4 + lg) * 16 + li] = make_float4(u0.x - p0[0], u0.y - p0[1], u0.z - p0[2], u0.w - p0[3]);
#pragma unroll
        for (int kk = 0; kk < NK; kk += 2) {
#define DR_STEP(E)                                           \
    y0 = dr_mfma1<E>(qf[kk], sf[kk], y0);                    \
    if (kk + 1 < NK) y1 = dr_mfma1<E>(qf[kk + 1], sf[kk + 1], y1);
            DR_EACH4(DR_STEP)
#undef DR_STEP
        }
        __builtin_amdgcn_sched_barrier(0);
        fetch_wq(cn);
        __builtin_amdgcn_sched_barrier(0);
        const float dec_now = dec;
        fetch_u(cn);
        __builtin_amdgcn_sched_barrier(0);
        __syncthreads();
        float4 uf[4];
#pragma unroll
        for (int kk = 0; kk < 4; ++kk) uf[kk] = Ul[(kk * 4 + lg) * 16 + li];
        __builtin_amdgcn_sched_barrier(0);
#pragma unroll
        for (int m = 0; m < NT; ++m) S[m] *= dec_now;
#pragma unroll
        for (int kk = 0; kk < 4; ++kk) {
#define DR_STEP(E)                                                                                  \
    _Pragma("unroll") for (int m = 0; m < NT; ++m) S[m] = dr_mfma1<E>(kf[m][kk], uf[kk], S[m]);      \
    y0 = dr_mfma1<E>(mf[kk], uf[kk], y0);
            DR_EACH4(DR_STEP)
#undef DR_STEP
        }
        const dr_f32x4 y = y0 + y1;
        __builtin_amdgcn_sched_barrier(0);
        fetch_k(cn);
        __builtin_amdgcn_sched_barrier(0);
        if (col_ok) {
            const int t = row0 + (c - c0) * DR_L + wave * 16 + 4 * lg;
#pragma unroll
            for (int e = 0; e < 4; ++e)
                if (t + e < row1) out[(size_t)(t + e) * ldo + (size_t)h * dv + j] = y[e];
        }
    }
#pragma unroll
    for (int m = 0; m < NT; ++m) {
        const int i = (wave + 4 * m) * 16 + 4 * lg;
#pragma unroll
        for (int e = 0; e < 4; ++e)
            if (col_ok && wave + 4 * m < NK && i + e < dk) st[i + e] = S[m][e];
    }
}

static int dr_padded_keys(int dk) { return dk <= 16 ? 16 : dk <= 32 ? 32 : dk <= 64 ? 64 : 128; }

extern "C" int tl_delta_chunked_takes(int dk, int dv) { return dk > 0 && dk <= 128 && dv > 0 ? 1 : 0; }
extern "C" int tl_delta_chunk_tokens() { return DR_L; }
// floats of workspace per chunk and head
extern "C" long long tl_delta_chunked_workspace(int dk, int dv) {
    const long long DP = dr_padded_keys(dk), DV = (dv + 15) / 16 * 16;
    return 3LL * DR_L * DP + DV * DR_L + DR_L * DR_L + 4;
}

// The operands of tl_delta_walk.  chunk_seq, chunk_row [NC]: a chunk's sequence and its first row of the step (a sequence's
// rows in chunks of DR_L from its first row on); seq_chunk [S + 1]: a sequence's first chunk (a sequence without chunks is
// left alone).  ws: NC * H *
// tl_delta_chunked_workspace floats, 16-byte aligned.
extern "C" int tl_delta_chunked(const float* q, int ldq, const float* k, int ldk, const float* v, int ldv, const float* b, int ldb,
                                const float* a, int lda, const float* rate_log, const float* step_bias, int share, float* state,
                                long long state_stride, const int32_t* state_slots, const int32_t* q_start,
                                const int32_t* chunk_seq, const int32_t* chunk_row, const int32_t* seq_chunk, float* ws, float* out,
                                int ldo, int S, int NC, int H, int dk, int dv, hipStream_t stream) {
    TL_CHECK_ARG(S >= 0 && NC >= 0 && H > 0 && tl_delta_chunked_takes(dk, dv),
                 "tl_delta_chunked: bad sizes S=%d H=%d dk=%d dv=%d", S, H, dk, dv);
    TL_CHECK_ARG(share >= 1 && H % share == 0, "tl_delta_chunked: %d heads do not share queries and keys in groups of %d", H, share);
    TL_CHECK_ARG(ldq >= H / share * dk && ldk >= H / share * dk && ldv >= H * dv && ldo >= H * dv && ldb >= H && lda >= H,
                 "tl_delta_chunked: rows too short");
    TL_CHECK_ARG(rate_log && state_stride >= (long long)H * dk * dv,
                 "tl_delta_chunked: rates are missing or the state of a request is too small");
    TL_CHECK_ARG(NC <= 65535 && H <= 65535 && S <= 65535, "tl_delta_chunked: too many chunks, heads or sequences for one launch");
    if (S == 0 || NC == 0) return 0;
    TL_CHECK_ARG(ws && (uintptr_t)ws % 16 == 0 && chunk_seq && chunk_row && seq_chunk,
                 "tl_delta_chunked: the workspace (16-byte aligned) or the chunk tables are missing");
    const int vec = ((uintptr_t)q % 16 == 0 && (uintptr_t)k % 16 == 0 && ldq % 4 == 0 && ldk % 4 == 0 && dk % 4 == 0) ? 1 : 0;
    const int DP = dr_padded_keys(dk), DV = (dv + 15) / 16 * 16;
    const size_t nh = (size_t)NC * H;
    float* ws_w = ws;
    float* ws_kt = ws_w + nh * DR_L * DP;
    float* ws_m = ws_kt + nh * DR_L * DP;
    float* ws_u0 = ws_m + nh * DR_L * DR_L;
    float* ws_q = ws_u0 + nh * DV * DR_L;
    float* ws_dec = ws_q + nh * DR_L * DP;
#define GO(NK)                                                                                                                     \
    do {                                                                                                                           \
        hipLaunchKernelGGL(delta_prepare_kernel<16 * NK>, dim3(H, NC), dim3(DR_THREADS), 0, stream, q, ldq, k, ldk, v, ldv, b, ldb, a, lda, \
                           rate_log, step_bias, share, q_start, chunk_seq, chunk_row, ws_u0, ws_w, ws_kt, ws_m, ws_q, ws_dec, H, dk, \
                           dv, vec);                                                                                                \
        TL_CHECK_LAUNCH("tl_delta_chunked prepare");                                                                               \
        hipLaunchKernelGGL(delta_states_kernel<NK>, dim3(H, tl_ceil_div(dv, 16), S), dim3(DR_THREADS), 0, stream, ws_u0, ws_w, ws_kt, ws_m, \
                           ws_q, ws_dec, state, state_stride, state_slots, q_start, seq_chunk, out, ldo, H, dk, dv);                  \
        TL_CHECK_LAUNCH("tl_delta_chunked states");                                                                                \
    } while (0)
    if (DP == 16) GO(1);
    else if (DP == 32) GO(2);
    else if (DP == 64) GO(4);
    else GO(8);
#undef GO
    return 0;
}
