// Residual branches joined to the stream with a factor, and the layer norm that reads the stream next, in one pass:
//
//     x[r] += mult * (y1[r] + y2[r])
//     out[r] = (x[r] - mean) / sqrt(mean((x[r] - mean)^2) + eps) * w + b
//
// y1 and y2 may each be absent, and each may come in shares (the K shares of a product, added in ascending order
// first).  With `rows`: out only, for the sums at rows[r]; x is left as it is.  Without w: the sum only.  Everything is
// float; the deviations are taken from the row's own mean, never from a difference of two large sums.
#include "common.h"

#define LN_VPT 4   // float4 per thread at most

__device__ __forceinline__ float4 ln_load4(const float* p) { return *reinterpret_cast<const float4*>(p); }
__device__ __forceinline__ void ln_store4(float* p, float4 v) { *reinterpret_cast<float4*>(p) = v; }
__device__ __forceinline__ void ln_store4(bf16_t* p, float4 v) {
    uint2 u;
    u.x = (uint32_t)tl_f2bf_bits(v.x) | ((uint32_t)tl_f2bf_bits(v.y) << 16);
    u.y = (uint32_t)tl_f2bf_bits(v.z) | ((uint32_t)tl_f2bf_bits(v.w) << 16);
    *reinterpret_cast<uint2*>(p) = u;
}

// A branch: null, or `parts` shares of it `stride` elements apart.
struct LnBranch {
    const float* y;
    int parts;
    long long stride;
};
__device__ __forceinline__ float ln_branch(const LnBranch& b, size_t i) {
    float v = b.y[i];
    for (int p = 1; p < b.parts; ++p) v += b.y[i + p * b.stride];
    return v;
}
__device__ __forceinline__ float4 ln_branch4(const LnBranch& b, size_t i) {
    float4 v = ln_load4(b.y + i);
    for (int p = 1; p < b.parts; ++p) {
        const float4 e = ln_load4(b.y + i + p * b.stride);
        v.x += e.x, v.y += e.y, v.z += e.z, v.w += e.w;
    }
    return v;
}

// Any row length: a thread walks its columns three times.
template <typename O>
__global__ __launch_bounds__(1024) void add_layernorm_kernel(float* __restrict__ x, LnBranch b1, LnBranch b2, float mult,
                                                             const float* __restrict__ w,
                                                             const float* __restrict__ b, float eps, O* __restrict__ out,
                                                             const int32_t* __restrict__ rows, int H) {
    __shared__ float red[16];
    const int r = blockIdx.x;
    const size_t src = rows ? (size_t)rows[r] : (size_t)r;
    float* xr = x + src * H;
    auto value = [&](int c) {
        float v = xr[c];
        if (b1.y) v += mult * (b2.y ? ln_branch(b1, src * H + c) + ln_branch(b2, src * H + c) : ln_branch(b1, src * H + c));
        return v;
    };
    float sum = 0.f;
    for (int c = threadIdx.x; c < H; c += blockDim.x) sum += value(c);
    sum = tl_block_sum(sum, red);
    const float mean = sum / (float)H;
    float ss = 0.f;
    for (int c = threadIdx.x; c < H; c += blockDim.x) {
        const float d = value(c) - mean;
        ss += d * d;
    }
    ss = tl_block_sum(ss, red);
    const float rstd = 1.0f / sqrtf(ss / (float)H + eps);
    for (int c = threadIdx.x; c < H; c += blockDim.x) {
        const float v = value(c);
        if (!rows && b1.y) xr[c] = v;
        if (w) out[(size_t)r * H + c] = tl_from_float<O>((v - mean) * rstd * w[c] + b[c]);
    }
}

// H a multiple of 4 and at most 16384: one pass over memory, 16-byte accesses, the row in registers meanwhile.
template <typename O>
__global__ __launch_bounds__(1024) void add_layernorm_vec_kernel(float* __restrict__ x, LnBranch b1, LnBranch b2, float mult,
                                                                 const float* __restrict__ w, const float* __restrict__ b, float eps,
                                                                 O* __restrict__ out, const int32_t* __restrict__ rows, int H) {
    __shared__ float red[16];
    const int r = blockIdx.x;
    const size_t src = rows ? (size_t)rows[r] : (size_t)r;
    float* xr = x + src * H;
    const int n4 = H >> 2;
    float4 v[LN_VPT];
    float sum = 0.f;
#pragma unroll
    for (int i = 0; i < LN_VPT; ++i) {
        const int c4 = threadIdx.x + i * blockDim.x;
        if (c4 < n4) {
            float4 a = ln_load4(xr + 4 * c4);
            if (b1.y) {
                float4 p = ln_branch4(b1, src * H + 4 * c4);
                if (b2.y) {
                    const float4 q = ln_branch4(b2, src * H + 4 * c4);
                    p.x += q.x, p.y += q.y, p.z += q.z, p.w += q.w;
                }
                a.x += mult * p.x, a.y += mult * p.y, a.z += mult * p.z, a.w += mult * p.w;
                if (!rows) ln_store4(xr + 4 * c4, a);
            }
            v[i] = a;
            sum += (a.x + a.y) + (a.z + a.w);
        }
    }
    if (!w) return;
    sum = tl_block_sum(sum, red);
    const float mean = sum / (float)H;
    float ss = 0.f;
#pragma unroll
    for (int i = 0; i < LN_VPT; ++i) {
        const int c4 = threadIdx.x + i * blockDim.x;
        if (c4 < n4) {
            v[i].x -= mean, v[i].y -= mean, v[i].z -= mean, v[i].w -= mean;
            ss += (v[i].x * v[i].x + v[i].y * v[i].y) + (v[i].z * v[i].z + v[i].w * v[i].w);
        }
    }
    ss = tl_block_sum(ss, red);
    const float rstd = 1.0f / sqrtf(ss / (float)H + eps);
    O* orow = out + (size_t)r * H;
#pragma unroll
    for (int i = 0; i < LN_VPT; ++i) {
        const int c4 = threadIdx.x + i * blockDim.x;
        if (c4 < n4) {
            const float4 g = ln_load4(w + 4 * c4), s = ln_load4(b + 4 * c4);
            float4 o;
            o.x = v[i].x * rstd * g.x + s.x;
            o.y = v[i].y * rstd * g.y + s.y;
            o.z = v[i].z * rstd * g.z + s.z;
            o.w = v[i].w * rstd * g.w + s.w;
            ln_store4(orow + 4 * c4, o);
        }
    }
}

// x float [n, H] (rows: [>= every row + 1, H]); y1, y2 float of x's shape or null (y2 only beside y1), in parts1 and parts2
// shares stride1 and stride2 elements apart; w, b float [H]
// and out [n_rows, H] float or bfloat16, or all three null: the sum only.
extern "C" int tl_add_layernorm(float* x, const float* y1, int parts1, long long stride1, const float* y2, int parts2,
                                long long stride2, float mult, const float* w, const float* b, float eps,
                                void* out, int out_dtype, const int32_t* rows, int n_rows, int H, hipStream_t stream) {
    TL_CHECK_ARG(n_rows >= 0 && H > 0 && eps >= 0.f, "tl_add_layernorm: bad sizes rows=%d H=%d", n_rows, H);
    TL_CHECK_ARG((w == nullptr) == (out == nullptr) && (w == nullptr) == (b == nullptr) && (rows == nullptr || w != nullptr),
                 "tl_add_layernorm: a norm needs weight, bias and output, and rows a norm");
    TL_CHECK_ARG(y1 || !y2, "tl_add_layernorm: a second branch without a first");
    TL_CHECK_ARG(parts1 >= 1 && parts1 <= 64 && parts2 >= 1 && parts2 <= 64 && (parts1 == 1 || stride1 > 0) && (parts2 == 1 || stride2 > 0),
                 "tl_add_layernorm: bad shares %d, %d", parts1, parts2);
    const LnBranch b1{y1, parts1, stride1}, b2{y2, parts2, stride2};
    if (n_rows == 0) return 0;
    const bool vec = H % 4 == 0 && H <= 1024 * 4 * LN_VPT && (parts1 == 1 || stride1 % 4 == 0) && (parts2 == 1 || stride2 % 4 == 0);
    int threads = (((vec ? H / 4 : H) + 63) / 64) * 64;
    if (threads > 1024) threads = 1024;
    if (vec && threads > 256 && n_rows >= 512) threads = H / 4 <= 256 * LN_VPT ? 256 : threads;   // many rows: several float4 per thread
    dim3 grid(n_rows), block(threads);
#define TL_LN(KERNEL, OT) hipLaunchKernelGGL(KERNEL<OT>, grid, block, 0, stream, x, b1, b2, mult, w, b, eps, (OT*)out, rows, H)
    if (out_dtype == TL_BF16) {
        if (vec) TL_LN(add_layernorm_vec_kernel, bf16_t);
        else TL_LN(add_layernorm_kernel, bf16_t);
    } else if (out_dtype == TL_F32) {
        if (vec) TL_LN(add_layernorm_vec_kernel, float);
        else TL_LN(add_layernorm_kernel, float);
    } else return tl_fail("tl_add_layernorm: unknown dtype %d", out_dtype);
#undef TL_LN
    TL_CHECK_LAUNCH("tl_add_layernorm");
    return 0;
}
