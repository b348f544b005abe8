// Several sublayers' results join the residual stream in one pass, each with a factor, and the
// norm that reads the stream next is applied on the way:
//     res[n, :] += sum_i f_i y_i[n, :]
//     out[n, :]  = norm(res[n, :])                                   (out null: none)
// A term y_i is float or bfloat16 [N, D], or the float partial sums [S, N, D] of a product whose
// S slices are still to be added; they are added in order, and the terms in order.  norm 0: the new
// rows themselves; 1: layer norm (x - mean) rsqrt(mean((x - mean)^2) + eps) w + b (b optional); 2: RMS
// norm x rsqrt(mean(x^2) + eps) w.  Float arithmetic, one rounding at the store of out.
#include "common.h"

#define TJ_MAX 4

struct TJTerms {
    const void* y[TJ_MAX];
    int bf16[TJ_MAX], slices[TJ_MAX];
    float factor[TJ_MAX];
    int n;
    size_t slice_stride;                          // elements of one slice: N * D
};

__device__ __forceinline__ float4 tj_load4(const float* p) { return *(const float4*)p; }
__device__ __forceinline__ float4 tj_load4(const bf16_t* p) {
    const uint2 r = *(const uint2*)p;
    return make_float4(__uint_as_float(r.x << 16), __uint_as_float(r.x & 0xffff0000u),
                       __uint_as_float(r.y << 16), __uint_as_float(r.y & 0xffff0000u));
}
__device__ __forceinline__ void tj_store4(float* p, float4 v) { *(float4*)p = v; }
__device__ __forceinline__ void tj_store4(bf16_t* p, float4 v) {
    uint2 r;
    r.x = (uint32_t)float_to_bf16(v.x) | ((uint32_t)float_to_bf16(v.y) << 16);
    r.y = (uint32_t)float_to_bf16(v.z) | ((uint32_t)float_to_bf16(v.w) << 16);
    *(uint2*)p = r;
}

// Any width and alignment: one workgroup per row, which goes through res twice more for the norm
// (every thread reads back only what it wrote).
template <typename T>
__global__ __launch_bounds__(256) void term_join_kernel(
        float* __restrict__ res, TJTerms t, int norm, const float* __restrict__ w,
        const float* __restrict__ b, float eps, T* __restrict__ out, int dim) {
    __shared__ float scratch[16];
    const size_t row = (size_t)blockIdx.x * dim;
    float sum = 0.f, sq = 0.f;
    for (int d = threadIdx.x; d < dim; d += 256) {
        float v = res[row + d];
        for (int i = 0; i < t.n; ++i) {
            float y = 0.f;
            if (t.bf16[i]) {
                y = load_as_float((const bf16_t*)t.y[i] + row + d);
            } else {
                for (int s = 0; s < t.slices[i]; ++s)
                    y += ((const float*)t.y[i])[s * t.slice_stride + row + d];
            }
            v = fmaf(t.factor[i], y, v);
        }
        res[row + d] = v;
        sum += v;
        sq = fmaf(v, v, sq);
    }
    if (!out) return;
    float mean = 0.f, rs = 1.f;
    if (norm == 1) {
        mean = block_sum(sum, scratch) / (float)dim;
        sq = 0.f;
        for (int d = threadIdx.x; d < dim; d += 256) {
            const float c = res[row + d] - mean;
            sq = fmaf(c, c, sq);
        }
    }
    if (norm) rs = rsqrtf(block_sum(sq, scratch) / (float)dim + eps);
    for (int d = threadIdx.x; d < dim; d += 256) {
        float v = (res[row + d] - mean) * rs;
        if (norm) v = v * w[d] + (b ? b[d] : 0.f);
        store_from_float(out + row + d, v);
    }
}

// Rows of up to THREADS * VPT * 4 elements, a multiple of 4, everything at multiples of 16 bytes:
// one pass over memory, the row stays in registers.
template <typename T, int VPT, int THREADS>
__global__ __launch_bounds__(THREADS) void term_join_vec_kernel(
        float* __restrict__ res, TJTerms t, int norm, const float* __restrict__ w,
        const float* __restrict__ b, float eps, T* __restrict__ out, int dim) {
    __shared__ float scratch[16];
    const size_t row = (size_t)blockIdx.x * dim;
    const int n4 = dim >> 2;
    float4 v[VPT];
    float sum = 0.f;
#pragma unroll
    for (int j = 0; j < VPT; ++j) {
        const int idx = threadIdx.x + j * THREADS;
        v[j] = make_float4(0.f, 0.f, 0.f, 0.f);
        if (idx >= n4) continue;
        const size_t at = row + 4 * (size_t)idx;
        v[j] = tj_load4(res + at);
        for (int i = 0; i < t.n; ++i) {
            float4 y;
            if (t.bf16[i]) {
                y = tj_load4((const bf16_t*)t.y[i] + at);
            } else {
                const float* src = (const float*)t.y[i] + at;
                y = tj_load4(src);
                for (int s = 1; s < t.slices[i]; ++s) {
                    const float4 a = tj_load4(src + s * t.slice_stride);
                    y.x += a.x; y.y += a.y; y.z += a.z; y.w += a.w;
                }
            }
            const float f = t.factor[i];
            v[j].x = fmaf(f, y.x, v[j].x);
            v[j].y = fmaf(f, y.y, v[j].y);
            v[j].z = fmaf(f, y.z, v[j].z);
            v[j].w = fmaf(f, y.w, v[j].w);
        }
        tj_store4(res + at, v[j]);
        sum += (v[j].x + v[j].y) + (v[j].z + v[j].w);
    }
    if (!out) return;
    float mean = 0.f, rs = 1.f;
    if (norm == 1) mean = block_sum(sum, scratch) / (float)dim;
    if (norm) {
        float sq = 0.f;
#pragma unroll
        for (int j = 0; j < VPT; ++j) {
            if (threadIdx.x + j * THREADS >= n4) continue;
            v[j].x -= mean; v[j].y -= mean; v[j].z -= mean; v[j].w -= mean;
            sq = fmaf(v[j].x, v[j].x, sq);
            sq = fmaf(v[j].y, v[j].y, sq);
            sq = fmaf(v[j].z, v[j].z, sq);
            sq = fmaf(v[j].w, v[j].w, sq);
        }
        rs = rsqrtf(block_sum(sq, scratch) / (float)dim + eps);
    }
#pragma unroll
    for (int j = 0; j < VPT; ++j) {
        const int idx = threadIdx.x + j * THREADS;
        if (idx >= n4) continue;
        float4 x = v[j];
        if (norm) {
            const float4 g = tj_load4(w + 4 * idx);
            const float4 c = b ? tj_load4(b + 4 * idx) : make_float4(0.f, 0.f, 0.f, 0.f);
            x = make_float4(x.x * rs * g.x + c.x, x.y * rs * g.y + c.y, x.z * rs * g.z + c.z,
                            x.w * rs * g.w + c.w);
        }
        tj_store4(out + row + 4 * (size_t)idx, x);
    }
}

template <typename T>
static int tj_launch(float* res, const TJTerms& t, int norm, const float* w, const float* b, float eps,
                     T* out, int n_rows, int dim, hipStream_t stream) {
    bool vec = dim % 4 == 0 && dim <= 8192 && (size_t)res % 16 == 0 && (size_t)w % 16 == 0
        && (size_t)b % 16 == 0 && (size_t)out % 16 == 0;
    for (int i = 0; i < t.n; ++i) vec = vec && (size_t)t.y[i] % 16 == 0;
#define TJ_ARGS res, t, norm, w, b, eps, out, dim
    if (!vec) term_join_kernel<T><<<n_rows, 256, 0, stream>>>(TJ_ARGS);
    else if (dim <= 1024) term_join_vec_kernel<T, 1, 256><<<n_rows, 256, 0, stream>>>(TJ_ARGS);
    else if (dim <= 4096) term_join_vec_kernel<T, 1, 1024><<<n_rows, 1024, 0, stream>>>(TJ_ARGS);
    else term_join_vec_kernel<T, 2, 1024><<<n_rows, 1024, 0, stream>>>(TJ_ARGS);
#undef TJ_ARGS
    return GFA_LAUNCH_RESULT();
}

extern "C" int gfa_term_join(float* res, const void* y0, const void* y1, const void* y2, const void* y3,
                             int n_terms, int bf16_mask, int s0, int s1, int s2, int s3, float f0, float f1,
                             float f2, float f3, int norm, const float* w, const float* b, float eps,
                             void* out, int out_bf16, int n_rows, int dim, hipStream_t stream) {
    if (n_rows <= 0) return 0;
    if (n_terms < 1 || n_terms > TJ_MAX || norm < 0 || norm > 2 || (out && norm && !w))
        return (int)hipErrorInvalidValue;
    TJTerms t{{y0, y1, y2, y3}, {}, {s0, s1, s2, s3}, {f0, f1, f2, f3}, n_terms, (size_t)n_rows * dim};
    for (int i = 0; i < TJ_MAX; ++i) {
        t.bf16[i] = (bf16_mask >> i) & 1;
        if (i < n_terms && (!t.y[i] || t.slices[i] < 1 || (t.bf16[i] && t.slices[i] != 1)))
            return (int)hipErrorInvalidValue;
    }
    if (out_bf16) return tj_launch<bf16_t>(res, t, norm, w, b, eps, (bf16_t*)out, n_rows, dim, stream);
    return tj_launch<float>(res, t, norm, w, b, eps, (float*)out, n_rows, dim, stream);
}
