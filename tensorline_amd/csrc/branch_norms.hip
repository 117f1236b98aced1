// Two residual branches with a scale per channel joined to the stream, and up to two RMS norms of the result, in one pass:
//
//     x[r] += scale1 * y1[r] + scale2 * y2[r]            (scales per channel, each may be absent)
//     out1[r] = x[r] / sqrt(mean(x[r]^2) + eps) * w1,    out2[r] = the same * w2
//
// A branch comes in pieces that are added in ascending order first: one piece (a plain [T, H] tensor), the K shares of a
// product ([P, T, H]), or the rows of a token's experts with a weight each ([T, top, H], weights [T, top]).  With `rows`: the
// norms of the sums at rows[r] only; x is left as it is.  Without w1: the sum only.  Everything is float.
#include "common.h"

#define BN_VPT 4   // float4 per thread at most

// piece p of token t starts at y + t * token + p * piece (null: no branch)
struct BnBranch {
    const float* y;
    int pieces;
    long long piece, token;
    const float* weights;     // [T, pieces] or null
    const float* scale;       // [H] or null
};

__device__ __forceinline__ float4 bn_load4(const float* p) { return *reinterpret_cast<const float4*>(p); }
__device__ __forceinline__ void bn_store4(float* p, float4 v) { *reinterpret_cast<float4*>(p) = v; }
__device__ __forceinline__ void bn_store4(bf16_t* p, float4 v) {
    uint2 u;
    u.x = (uint32_t)tl_f2bf_bits(v.x) | ((uint32_t)tl_f2bf_bits(v.y) << 16);
    u.y = (uint32_t)tl_f2bf_bits(v.z) | ((uint32_t)tl_f2bf_bits(v.w) << 16);
    *reinterpret_cast<uint2*>(p) = u;
}

__device__ __forceinline__ float bn_branch(const BnBranch& b, size_t t, int c) {
    const float* y = b.y + t * b.token + c;
    float v;
    if (b.weights) {
        v = 0.f;
        for (int p = 0; p < b.pieces; ++p) v = __builtin_fmaf(b.weights[t * b.pieces + p], y[p * b.piece], v);
    } else {
        v = y[0];
        for (int p = 1; p < b.pieces; ++p) v += y[p * b.piece];
    }
    return b.scale ? v * b.scale[c] : v;
}
__device__ __forceinline__ float4 bn_branch4(const BnBranch& b, size_t t, int c) {
    const float* y = b.y + t * b.token + c;
    float4 v;
    if (b.weights) {
        v = make_float4(0.f, 0.f, 0.f, 0.f);
        for (int p = 0; p < b.pieces; ++p) {
            const float w = b.weights[t * b.pieces + p];
            const float4 e = bn_load4(y + p * b.piece);
            v.x = __builtin_fmaf(w, e.x, v.x), v.y = __builtin_fmaf(w, e.y, v.y);
            v.z = __builtin_fmaf(w, e.z, v.z), v.w = __builtin_fmaf(w, e.w, v.w);
        }
    } else {
        v = bn_load4(y);
        for (int p = 1; p < b.pieces; ++p) {
            const float4 e = bn_load4(y + p * b.piece);
            v.x += e.x, v.y += e.y, v.z += e.z, v.w += e.w;
        }
    }
    if (b.scale) {
        const float4 m = bn_load4(b.scale + c);
        v.x *= m.x, v.y *= m.y, v.z *= m.z, v.w *= m.w;
    }
    return v;
}

// Any row length: a thread walks its columns twice.
template <typename O>
__global__ __launch_bounds__(1024) void join_norms_kernel(float* __restrict__ x, BnBranch b1, BnBranch b2, const float* __restrict__ w1,
                                                          const float* __restrict__ w2, float eps, O* __restrict__ out1,
                                                          O* __restrict__ out2, const int32_t* __restrict__ rows, int H) {
    __shared__ float red[16];
    const int r = blockIdx.x;
    const size_t src = rows ? (size_t)rows[r] : (size_t)r;
    float* xr = x + src * H;
    auto value = [&](int c) {
        float v = xr[c];
        if (b1.y) {
            float y = bn_branch(b1, src, c);
            if (b2.y) y += bn_branch(b2, src, c);
            v += y;
        }
        return v;
    };
    float ss = 0.f;
    for (int c = threadIdx.x; c < H; c += blockDim.x) {
        const float v = value(c);
        ss += v * v;
    }
    float rstd = 0.f;
    if (w1) {
        ss = tl_block_sum(ss, red);
        rstd = 1.0f / sqrtf(ss / (float)H + eps);
    }
    for (int c = threadIdx.x; c < H; c += blockDim.x) {
        const float v = value(c);
        if (!rows && b1.y) xr[c] = v;
        if (w1) out1[(size_t)r * H + c] = tl_from_float<O>(v * rstd * w1[c]);
        if (w2) out2[(size_t)r * H + c] = tl_from_float<O>(v * rstd * w2[c]);
    }
}

// H a multiple of 4 and at most 16384: one pass over memory, 16-byte accesses, the row in registers meanwhile.
template <typename O>
__global__ __launch_bounds__(1024) void join_norms_vec_kernel(float* __restrict__ x, BnBranch b1, BnBranch b2, const float* __restrict__ w1,
                                                              const float* __restrict__ w2, float eps, O* __restrict__ out1,
                                                              O* __restrict__ out2, const int32_t* __restrict__ rows, int H) {
    __shared__ float red[16];
    const int r = blockIdx.x;
    const size_t src = rows ? (size_t)rows[r] : (size_t)r;
    float* xr = x + src * H;
    const int n4 = H >> 2;
    float4 v[BN_VPT];
    float ss = 0.f;
#pragma unroll
    for (int i = 0; i < BN_VPT; ++i) {
        const int c4 = threadIdx.x + i * blockDim.x;
        if (c4 < n4) {
            float4 a = bn_load4(xr + 4 * c4);
            if (b1.y) {
                float4 p = bn_branch4(b1, src, 4 * c4);
                if (b2.y) {
                    const float4 q = bn_branch4(b2, src, 4 * c4);
                    p.x += q.x, p.y += q.y, p.z += q.z, p.w += q.w;
                }
                a.x += p.x, a.y += p.y, a.z += p.z, a.w += p.w;
                if (!rows) bn_store4(xr + 4 * c4, a);
            }
            v[i] = a;
            ss += (a.x * a.x + a.y * a.y) + (a.z * a.z + a.w * a.w);
        }
    }
    if (!w1) return;
    ss = tl_block_sum(ss, red);
    const float rstd = 1.0f / sqrtf(ss / (float)H + eps);
#pragma unroll
    for (int i = 0; i < BN_VPT; ++i) {
        const int c4 = threadIdx.x + i * blockDim.x;
        if (c4 < n4) {
            const float4 n = make_float4(v[i].x * rstd, v[i].y * rstd, v[i].z * rstd, v[i].w * rstd);
            const float4 g = bn_load4(w1 + 4 * c4);
            bn_store4(out1 + (size_t)r * H + 4 * c4, make_float4(n.x * g.x, n.y * g.y, n.z * g.z, n.w * g.w));
            if (w2) {
                const float4 m = bn_load4(w2 + 4 * c4);
                bn_store4(out2 + (size_t)r * H + 4 * c4, make_float4(n.x * m.x, n.y * m.y, n.z * m.z, n.w * m.w));
            }
        }
    }
}

// x float [n, H] (rows: [>= every row + 1, H]); y1, y2 or null (y2 only beside y1); scale1, scale2, w1, w2 float [H] or null; out1,
// out2 [n_rows, H] float or bfloat16, null exactly where w1, w2 are.
extern "C" int tl_join_norms(float* x, const float* y1, int pieces1, long long piece1, long long token1, const float* weights1,
                             const float* scale1, const float* y2, int pieces2, long long piece2, long long token2, const float* weights2,
                             const float* scale2, const float* w1, const float* w2, float eps, void* out1, void* out2, int out_dtype,
                             const int32_t* rows, int n_rows, int H, hipStream_t stream) {
    TL_CHECK_ARG(n_rows >= 0 && H > 0 && eps >= 0.f, "tl_join_norms: bad sizes rows=%d H=%d", n_rows, H);
    TL_CHECK_ARG((w1 == nullptr) == (out1 == nullptr) && (w2 == nullptr) == (out2 == nullptr) && (w1 || !w2) && (!rows || w1),
                 "tl_join_norms: a norm needs weight and output, a second norm a first, and rows a norm");
    TL_CHECK_ARG(y1 || !y2, "tl_join_norms: a second branch without a first");
    TL_CHECK_ARG(!y1 || (pieces1 >= 1 && pieces1 <= 64 && token1 >= H && (pieces1 == 1 || piece1 >= H)), "tl_join_norms: bad pieces %d of the first branch", pieces1);
    TL_CHECK_ARG(!y2 || (pieces2 >= 1 && pieces2 <= 64 && token2 >= H && (pieces2 == 1 || piece2 >= H)), "tl_join_norms: bad pieces %d of the second branch", pieces2);
    const BnBranch b1{y1, pieces1, piece1, token1, weights1, scale1}, b2{y2, pieces2, piece2, token2, weights2, scale2};
    if (n_rows == 0) return 0;
    auto aligned = [](const void* p) { return (uintptr_t)p % 16 == 0; };
    const bool vec = H % 4 == 0 && H <= 1024 * 4 * BN_VPT && aligned(x) && aligned(y1) && aligned(y2) && aligned(scale1) && aligned(scale2) &&
                     aligned(w1) && aligned(w2) && aligned(out1) && aligned(out2) && piece1 % 4 == 0 && token1 % 4 == 0 && piece2 % 4 == 0 && token2 % 4 == 0;
    int threads = (((vec ? H / 4 : H) + 63) / 64) * 64;
    if (threads > 1024) threads = 1024;
    if (vec && threads > 256 && n_rows >= 512) threads = H / 4 <= 256 * BN_VPT ? 256 : threads;   // many rows: several float4 per thread
    dim3 grid(n_rows), block(threads);
#define GO(KERNEL, OT) hipLaunchKernelGGL(KERNEL<OT>, grid, block, 0, stream, x, b1, b2, w1, w2, eps, (OT*)out1, (OT*)out2, rows, H)
    if (out_dtype == TL_BF16) {
        if (vec) GO(join_norms_vec_kernel, bf16_t);
        else GO(join_norms_kernel, bf16_t);
    } else if (out_dtype == TL_F32) {
        if (vec) GO(join_norms_vec_kernel, float);
        else GO(join_norms_kernel, float);
    } else return tl_fail("tl_join_norms: unknown dtype %d", out_dtype);
#undef GO
    TL_CHECK_LAUNCH("tl_join_norms");
    return 0;
}

// ---- RMS norm of rows that are a block of columns of a wider float matrix -----------------------------------------
template <typename O>
__global__ __launch_bounds__(256) void norm_rows_kernel(const float* __restrict__ x, int ldx, const float* __restrict__ w, float eps,
                                                        O* __restrict__ out, int n) {
    __shared__ float red[16];
    const float* row = x + (size_t)blockIdx.x * ldx;
    float ss = 0.f;
    for (int c = threadIdx.x; c < n; c += blockDim.x) ss += row[c] * row[c];
    ss = tl_block_sum(ss, red);
    const float rstd = 1.0f / sqrtf(ss / (float)n + eps);
    for (int c = threadIdx.x; c < n; c += blockDim.x) out[(size_t)blockIdx.x * n + c] = tl_from_float<O>(row[c] * rstd * w[c]);
}

extern "C" int tl_norm_rows(const float* x, int ldx, const float* w, float eps, void* out, int out_dtype, int T, int n, hipStream_t stream) {
    TL_CHECK_ARG(T >= 0 && n > 0 && ldx >= n && x && w && out && eps >= 0.f, "tl_norm_rows: bad sizes T=%d n=%d", T, n);
    if (T == 0) return 0;
    const dim3 block(n >= 256 ? 256 : 64 * tl_ceil_div(n, 64));
    if (out_dtype == TL_BF16) hipLaunchKernelGGL(norm_rows_kernel<bf16_t>, dim3(T), block, 0, stream, x, ldx, w, eps, (bf16_t*)out, n);
    else if (out_dtype == TL_F32) hipLaunchKernelGGL(norm_rows_kernel<float>, dim3(T), block, 0, stream, x, ldx, w, eps, (float*)out, n);
    else return tl_fail("tl_norm_rows: unknown dtype %d", out_dtype);
    TL_CHECK_LAUNCH("tl_norm_rows");
    return 0;
}

// ---- logits scaled and bent by a cap, in place: z <- cap tanh(scale z / cap); cap 0: z <- scale z ---------------------
__global__ __launch_bounds__(256) void scale_cap_kernel(float* __restrict__ z, long long n, float scale, float cap) {
    const long long i = (long long)blockIdx.x * blockDim.x + threadIdx.x;
    if (i >= n) return;
    const float v = z[i] * scale;
    z[i] = cap > 0.f ? cap * tanhf(v / cap) : v;
}

extern "C" int tl_scale_cap(float* z, long long n, float scale, float cap, hipStream_t stream) {
    TL_CHECK_ARG(n >= 0 && z && cap >= 0.f, "tl_scale_cap: bad sizes or a negative cap");
    if (n == 0) return 0;
    TL_CHECK_ARG((n + 255) / 256 <= 0x7fffffffLL, "tl_scale_cap: too many values");
    hipLaunchKernelGGL(scale_cap_kernel, dim3((unsigned)((n + 255) / 256)), dim3(256), 0, stream, z, n, scale, cap);
    TL_CHECK_LAUNCH("tl_scale_cap");
    return 0;
}
