// The selective scan of Mamba (Gu and Dao, "Mamba: Linear-Time Sequence Modeling with Selective State Spaces"): for
// each channel, with vectors over its N states and the channel's own dt = softplus(dt_raw + dt_bias), x, z at token t,
//
//     S_t = exp(dt_t A) S_(t-1) + (dt_t x_t) B_t,   out_t = (C_t . S_t + D x_t) silu(z_t)
//
// S of a request is kept in its slot between steps, [state n][channel].  All arithmetic is float; A comes times log2 e, so
// that a decay is one v_exp_f32.
//
// A lane owns up to R states of one channel in registers; a channel with more is spread over P lanes of a wave, P a power of
// two, whose shares of y are added by lane exchanges.  Neighbouring lanes own neighbouring channels, so every access but
// that of B and C (through LDS, the same for all channels) is a run of consecutive floats.
//
// Decode steps and short portions walk a sequence's tokens in one launch.  Longer portions are cut into chunks of SS_L tokens
// from a sequence's first row of the step: a state's decay over a chunk is exp(A sum dt), so
//   1. scan_kernel<LOCAL> gives every chunk's own contribution to the state (from zero) and its sums of dt, all chunks at once,
//      and leaves dt in place of dt_raw;
//   2. scan_states_kernel walks the chunks per state and leaves what enters each of them in place of its own contribution;
//   3. scan_kernel<OUTPUT> takes every chunk from the state that enters it; a sequence's last chunk renews its slot.
// Tokens within a chunk are taken in order by the same instructions in every form, so results agree across cuttings within
// rounding.
#include "common.h"

#include <math.h>

#define SS_L 64            // tokens per chunk
#define SS_TT 16           // tokens whose B and C lie in LDS at a time
#define SS_AHEAD 8         // tokens whose per-channel operands are loaded together
#define SS_MAX_STATE 256
#define SS_THREADS 256

#define SS_LOG2E 1.4426950408889634f
#define SS_LN2 0.6931471805599453f
// softplus(z) = max(z, 0) + ln(1 + w), w = exp(-|z|): ln(1 + w) = ln(u) w / (u - 1) with u the float nearest 1 + w, which takes
// out what rounding 1 + w lost; w itself where u is 1
__device__ __forceinline__ float ss_softplus(float z) {
    const float w = __builtin_amdgcn_exp2f(-SS_LOG2E * fabsf(z)), u = 1.0f + w, d = u - 1.0f;
    const float l = d == 0.f ? w : SS_LN2 * __builtin_amdgcn_logf(u) * (w * __builtin_amdgcn_rcpf(d));
    return fmaxf(z, 0.f) + l;
}
__device__ __forceinline__ float ss_silu(float z) { return z * __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(-SS_LOG2E * z)); }

enum { SS_WALK = 0, SS_LOCAL = 1, SS_OUTPUT = 2 };

// X: the storage type of x and of the output.  dt_raw float [T, >= inner], z float [T, >= inner], bc float [T, >= 2 N]
// = [B | C]; A2 float [N][inner].
template <int R, int P, int MODE, typename X>
__global__ __launch_bounds__(SS_THREADS) void scan_kernel(
    float* __restrict__ dt_raw, int lddt, const float* __restrict__ dt_bias, const X* __restrict__ x, int ldx,
    const float* __restrict__ z, int ldz, const float* __restrict__ bc, int ldbc, const float* __restrict__ A2,
    const float* __restrict__ D, float* __restrict__ state, long long state_stride, const int32_t* __restrict__ state_slots,
    const int32_t* __restrict__ q_start, const int32_t* __restrict__ chunk_seq, const int32_t* __restrict__ chunk_row,
    float* __restrict__ ws_state, float* __restrict__ ws_dt, X* __restrict__ out, int ldo, int inner, int N, int upto) {
    constexpr int NP = R * P, CW = 64 / P, CB = SS_THREADS / P;
    __shared__ __attribute__((aligned(16))) float Bs[SS_TT][NP], Cs[MODE == SS_LOCAL ? 1 : SS_TT][NP];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const int p = lane / CW, ch = blockIdx.x * CB + wave * CW + lane % CW;
    const bool ch_ok = ch < inner;
    const int cc = ch_ok ? ch : inner - 1;
    int s, t0, t1;
    if (MODE == SS_WALK) {
        s = blockIdx.y;
        t0 = q_start[s];
        t1 = q_start[s + 1];
        if (t1 <= t0 || t1 - t0 > upto) return;
    } else {
        s = chunk_seq[blockIdx.y];
        t0 = chunk_row[blockIdx.y];
        t1 = q_start[s + 1];
        if (MODE == SS_LOCAL && t1 - t0 <= SS_L) {                // nothing follows a sequence's last chunk: its steps only
            if (p == 0 && ch_ok) {
                const float bias = dt_bias ? dt_bias[ch] : 0.f;
                for (int t = t0; t < t1; ++t) dt_raw[(size_t)t * lddt + ch] = ss_softplus(dt_raw[(size_t)t * lddt + ch] + bias);
            }
            return;
        }
        if (t1 - t0 > SS_L) t1 = t0 + SS_L;
    }
    const bool last = MODE != SS_LOCAL && t1 == q_start[s + 1];
    float* slot = state + (size_t)state_slots[s] * state_stride;
    float* mine = MODE == SS_WALK ? slot : ws_state + (size_t)blockIdx.y * N * inner;
    float S[R], a2[R];
#pragma unroll
    for (int r = 0; r < R; ++r) {
        const int n = p * R + r;
        a2[r] = n < N ? A2[(size_t)n * inner + cc] : 0.f;
        S[r] = (MODE != SS_LOCAL && n < N) ? mine[(size_t)n * inner + cc] : 0.f;
    }
    const float bias = dt_bias ? dt_bias[cc] : 0.f, skip = MODE == SS_LOCAL ? 0.f : D[cc];
    float sum_dt = 0.f;
    for (int tb = t0; tb < t1; tb += SS_TT) {
        if (tb > t0) __syncthreads();                             // the tile before is used up
        for (int idx = tid; idx < SS_TT * NP; idx += SS_THREADS) {
            const int tt = idx / NP, n = idx % NP;
            const bool ok = tb + tt < t1 && n < N;
            const float* row = bc + (size_t)(tb + tt) * ldbc;
            Bs[tt][n] = ok ? row[n] : 0.f;
            if (MODE != SS_LOCAL) Cs[tt][n] = ok ? row[N + n] : 0.f;
        }
        __syncthreads();
#pragma unroll
        for (int ta = 0; ta < SS_TT; ta += SS_AHEAD) {
            if (tb + ta >= t1) break;
            float xv[SS_AHEAD], dv[SS_AHEAD], zv[MODE == SS_LOCAL ? 1 : SS_AHEAD];
#pragma unroll
            for (int u = 0; u < SS_AHEAD; ++u) {
                const int t = tb + ta + u < t1 ? tb + ta + u : t1 - 1;
                xv[u] = tl_to_float(x[(size_t)t * ldx + cc]);
                dv[u] = dt_raw[(size_t)t * lddt + cc];
                if (MODE != SS_LOCAL) zv[u] = z[(size_t)t * ldz + cc];
            }
#pragma unroll
            for (int u = 0; u < SS_AHEAD; ++u) {
                const int tt = ta + u, t = tb + tt;
                if (t >= t1) break;
                const float dt = MODE == SS_OUTPUT ? dv[u] : ss_softplus(dv[u] + bias), dx = dt * xv[u];
                if (MODE == SS_LOCAL) {
                    sum_dt += dt;
                    if (p == 0 && ch_ok) dt_raw[(size_t)t * lddt + ch] = dt;
                }
                float y0 = 0.f, y1 = 0.f;
#pragma unroll
                for (int r4 = 0; r4 < R; r4 += 4) {
                    const float4 Bv = *reinterpret_cast<const float4*>(&Bs[tt][p * R + r4]);
                    float4 Cv = make_float4(0.f, 0.f, 0.f, 0.f);
                    if (MODE != SS_LOCAL) Cv = *reinterpret_cast<const float4*>(&Cs[tt][p * R + r4]);
#define SS_STATE(E, BV, CV, Y)                                                                    \
    S[r4 + E] = __builtin_fmaf(__builtin_amdgcn_exp2f(dt * a2[r4 + E]), S[r4 + E], dx * BV);      \
    if (MODE != SS_LOCAL) Y = __builtin_fmaf(S[r4 + E], CV, Y);
                    SS_STATE(0, Bv.x, Cv.x, y0)
                    SS_STATE(1, Bv.y, Cv.y, y1)
                    SS_STATE(2, Bv.z, Cv.z, y0)
                    SS_STATE(3, Bv.w, Cv.w, y1)
#undef SS_STATE
                }
                if (MODE != SS_LOCAL) {
                    float y = y0 + y1;
#pragma unroll
                    for (int off = CW; off < 64; off <<= 1) y += __shfl_xor(y, off, TL_WAVE);
                    y = __builtin_fmaf(skip, xv[u], y);
                    if (p == 0 && ch_ok) out[(size_t)t * ldo + ch] = tl_from_float<X>(y * ss_silu(zv[u]));
                }
            }
        }
    }
    if (!ch_ok) return;
    if (MODE == SS_LOCAL || last) {
        float* dst = MODE == SS_LOCAL ? mine : slot;
#pragma unroll
        for (int r = 0; r < R; ++r) {
            const int n = p * R + r;
            if (n < N) dst[(size_t)n * inner + ch] = S[r];
        }
    }
    if (MODE == SS_LOCAL && p == 0) ws_dt[(size_t)blockIdx.y * inner + ch] = sum_dt;
}

// Per state element, the chunks of a sequence in order: what enters each chunk is left in the workspace.
__global__ __launch_bounds__(SS_THREADS) void scan_states_kernel(float* __restrict__ ws_state, const float* __restrict__ ws_dt,
                                                                 const float* __restrict__ A2, const float* __restrict__ state,
                                                                 long long state_stride, const int32_t* __restrict__ state_slots,
                                                                 const int32_t* __restrict__ seq_chunk, int inner, int N) {
    const int ch = blockIdx.x * SS_THREADS + threadIdx.x, n = blockIdx.y, s = blockIdx.z;
    if (ch >= inner) return;
    const int c0 = seq_chunk[s], c1 = seq_chunk[s + 1];
    if (c1 <= c0) return;
    const float a2 = A2[(size_t)n * inner + ch];
    float S = state[(size_t)state_slots[s] * state_stride + (size_t)n * inner + ch];
    float* w = ws_state + (size_t)n * inner + ch;
    const size_t step = (size_t)N * inner;
    for (int c = c0; c < c1; c += 8) {
        float own[8], dt[8];
#pragma unroll
        for (int u = 0; u < 8; ++u) {                             // the last chunk has no contribution of its own here
            const int cu = c + u < c1 - 1 ? c + u : c0;
            own[u] = w[(size_t)cu * step];
            dt[u] = ws_dt[(size_t)cu * inner + ch];
        }
#pragma unroll
        for (int u = 0; u < 8; ++u) {
            if (c + u >= c1) break;
            w[(size_t)(c + u) * step] = S;
            if (c + u < c1 - 1) S = __builtin_fmaf(__builtin_amdgcn_exp2f(dt[u] * a2), S, own[u]);
        }
    }
}

extern "C" int tl_selective_scan_takes(int N) { return N > 0 && N <= SS_MAX_STATE ? 1 : 0; }
extern "C" int tl_selective_scan_chunk_tokens() { return SS_L; }

template <int MODE, typename X>
static int ss_launch(float* dt_raw, int lddt, const float* dt_bias, const void* x, int ldx, const float* z, int ldz,
                     const float* bc, int ldbc, const float* A2, const float* D, float* state, long long state_stride,
                     const int32_t* state_slots, const int32_t* q_start, const int32_t* chunk_seq, const int32_t* chunk_row,
                     float* ws_state, float* ws_dt, void* out, int ldo, int rows, int inner, int N, int upto,
                     hipStream_t stream) {
#define GO(R, P)                                                                                                                      \
    hipLaunchKernelGGL((scan_kernel<R, P, MODE, X>), dim3(tl_ceil_div(inner, SS_THREADS / P), rows), dim3(SS_THREADS), 0, stream, dt_raw, \
                       lddt, dt_bias, (const X*)x, ldx, z, ldz, bc, ldbc, A2, D, state, state_stride, state_slots, q_start, chunk_seq, \
                       chunk_row, ws_state, ws_dt, (X*)out, ldo, inner, N, upto)
    if (N <= 8) GO(8, 1);
    else if (N <= 16) GO(16, 1);
    else if (N <= 32) GO(16, 2);
    else if (N <= 64) GO(16, 4);
    else if (N <= 128) GO(16, 8);
    else GO(16, 16);
#undef GO
    TL_CHECK_LAUNCH("tl_selective_scan");
    return 0;
}

// dt_raw (overwritten where NC > 0), z float [T, >= inner], bc float [T, >= 2 N] = [B | C], x and out [T, >= inner] of
// dtype; dt_bias [inner] or null, A2 [N, inner] = A log2 e, D [inner]; state: a request's [N, inner] at
// state + slot * state_stride.  NC = 0: every sequence's tokens are walked in order.  Else chunk_seq, chunk_row [NC], seq_chunk [S + 1] (chunks of SS_L tokens from a sequence's
// first row of the step on; a sequence without chunks is left to the walk), ws_state NC * N * inner floats, ws_dt NC * inner
// floats; walk_upto > 0: the sequences that bring at most so many rows are walked beside them.
extern "C" int tl_selective_scan(float* dt_raw, int lddt, const float* dt_bias, const void* x, int ldx, const float* z, int ldz,
                                 const float* bc, int ldbc, const float* A2, const float* D, float* state, long long state_stride,
                                 const int32_t* state_slots, const int32_t* q_start, const int32_t* chunk_seq,
                                 const int32_t* chunk_row, const int32_t* seq_chunk, float* ws_state, float* ws_dt, void* out,
                                 int dtype, int ldo, int S, int NC, int inner, int N, int walk_upto, hipStream_t stream) {
    TL_CHECK_ARG(S >= 0 && NC >= 0 && inner > 0 && tl_selective_scan_takes(N),
                 "tl_selective_scan: bad sizes inner=%d state=%d (at most %d)", inner, N, SS_MAX_STATE);
    TL_CHECK_ARG(lddt >= inner && ldx >= inner && ldz >= inner && ldo >= inner && ldbc >= 2 * N, "tl_selective_scan: rows too short");
    TL_CHECK_ARG(A2 && D && state_stride >= (long long)N * inner,
                 "tl_selective_scan: A or D is missing, or the state of a request is too small");
    TL_CHECK_ARG(S <= 65535 && NC <= 65535, "tl_selective_scan: too many sequences or chunks for one launch");
    TL_CHECK_ARG(dtype == TL_F32 || dtype == TL_BF16, "tl_selective_scan: unknown dtype %d", dtype);
    if (S == 0) return 0;
#define GO(MODE, ROWS)                                                                                                              \
    (dtype == TL_BF16 ? ss_launch<MODE, bf16_t>(dt_raw, lddt, dt_bias, x, ldx, z, ldz, bc, ldbc, A2, D, state, state_stride, state_slots, \
                                                q_start, chunk_seq, chunk_row, ws_state, ws_dt, out, ldo, ROWS, inner, N, walk_upto, stream)    \
                      : ss_launch<MODE, float>(dt_raw, lddt, dt_bias, x, ldx, z, ldz, bc, ldbc, A2, D, state, state_stride, state_slots, \
                                               q_start, chunk_seq, chunk_row, ws_state, ws_dt, out, ldo, ROWS, inner, N, walk_upto, stream))
    if (NC == 0 || walk_upto > 0) {
        if (NC == 0) walk_upto = 0x7fffffff;
        const int rc = GO(SS_WALK, S);
        if (rc || NC == 0) return rc;
    }
    TL_CHECK_ARG(chunk_seq && chunk_row && seq_chunk && ws_state && ws_dt, "tl_selective_scan: chunk tables or workspace are missing");
    if (int rc = GO(SS_LOCAL, NC)) return rc;
    hipLaunchKernelGGL(scan_states_kernel, dim3(tl_ceil_div(inner, SS_THREADS), N, S), dim3(SS_THREADS), 0, stream, ws_state, ws_dt, A2,
                       state, state_stride, state_slots, seq_chunk, inner, N);
    TL_CHECK_LAUNCH("tl_selective_scan states");
    return GO(SS_OUTPUT, NC);
#undef GO
}
