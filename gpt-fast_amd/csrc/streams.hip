// Several residual streams in place of one (hyper-connections): X [n_tokens, S, dim], float.
//     read:  u = sum_s in[s] X_s;   out = u * rsqrt(mean(u^2) + eps) * w          (type T)
//     join:  X_t <- sum_s mix[s, t] X_s + outw[t] y, all streams from the old ones, and the read
//            that comes next (of the new streams) in the same pass
// y is what a sublayer gave: float or bfloat16 rows, or float partial sums of a sliced product
// (n_parts of them, added in order).  One workgroup per token, sums and statistics in float, one
// rounding at the store.  The order of additions depends on the row alone.
#include "common.h"

#define ST_MAX 16                       // streams

struct STMix {
    const float* mix;                   // [S, S], from the row's stream to the column's
    const float* outw;                  // [S]
    const float* in;                    // [S], the next read; null: none
};

__global__ void streams_spread_kernel(const float* __restrict__ x, float* __restrict__ X, int S, int dim) {
    const float* row = x + (size_t)blockIdx.x * dim;
    float* o = X + (size_t)blockIdx.x * S * dim;
    for (int d = threadIdx.x; d < dim; d += blockDim.x) {
        const float v = row[d];
        for (int s = 0; s < S; ++s) o[(size_t)s * dim + d] = v;
    }
}

extern "C" int gfa_streams_spread(const float* x, float* X, int n_rows, int S, int dim, hipStream_t stream) {
    if (n_rows <= 0) return 0;
    if (S < 1 || S > ST_MAX) return (int)hipErrorInvalidValue;
    streams_spread_kernel<<<n_rows, dim > 1024 ? 1024 : 256, 0, stream>>>(x, X, S, dim);
    return GFA_LAUNCH_RESULT();
}

template <typename Y> __device__ __forceinline__ float4 st_load4(const Y* p);
template <> __device__ __forceinline__ float4 st_load4<float>(const float* p) { return *(const float4*)p; }
template <> __device__ __forceinline__ float4 st_load4<bf16_t>(const bf16_t* p) {
    const uint2 v = *(const uint2*)p;
    return make_float4(__uint_as_float(v.x << 16), __uint_as_float(v.x & 0xffff0000u),
                       __uint_as_float(v.y << 16), __uint_as_float(v.y & 0xffff0000u));
}
__device__ __forceinline__ void st_store4(float* p, float4 v) { *(float4*)p = v; }
__device__ __forceinline__ void st_store4(bf16_t* p, float4 v) {
    *(uint2*)p = make_uint2((uint32_t)float_to_bf16(v.x) | ((uint32_t)float_to_bf16(v.y) << 16),
                            (uint32_t)float_to_bf16(v.z) | ((uint32_t)float_to_bf16(v.w) << 16));
}
__device__ __forceinline__ float4 st_fma(float a, float4 x, float4 c) {
    return make_float4(fmaf(a, x.x, c.x), fmaf(a, x.y, c.y), fmaf(a, x.z, c.z), fmaf(a, x.w, c.w));
}

// Any size: the elements of a row are walked one by one.  JOIN 0: read only (row rows ? rows[i] : i).
template <typename T, typename Y, int JOIN>
__global__ __launch_bounds__(256) void streams_kernel(
        float* __restrict__ X, const Y* __restrict__ y, int n_parts, size_t part_stride, STMix m,
        const float* __restrict__ w, float eps, const int* __restrict__ rows, T* __restrict__ out, int S,
        int dim) {
    __shared__ float scratch[16];
    const int i = blockIdx.x;
    float* x = X + (size_t)(rows ? rows[i] : i) * S * dim;
    float ss = 0.f;
    for (int d = threadIdx.x; d < dim; d += 256) {
        float old[ST_MAX], u = 0.f;
#pragma unroll
        for (int s = 0; s < ST_MAX; ++s) old[s] = s < S ? x[(size_t)s * dim + d] : 0.f;
        if (JOIN) {
            float yv = load_as_float(y + (size_t)i * dim + d);
            for (int p = 1; p < n_parts; ++p) yv += load_as_float(y + p * part_stride + (size_t)i * dim + d);
            for (int t = 0; t < S; ++t) {
                float v = m.outw[t] * yv;
#pragma unroll
                for (int s = 0; s < ST_MAX; ++s)
                    if (s < S) v = fmaf(m.mix[s * S + t], old[s], v);
                x[(size_t)t * dim + d] = v;
                if (m.in) u = fmaf(m.in[t], v, u);
            }
        } else {
#pragma unroll
            for (int s = 0; s < ST_MAX; ++s)
                if (s < S) u = fmaf(m.in[s], old[s], u);
        }
        ss = fmaf(u, u, ss);
    }
    if (!m.in) return;
    const float r = rsqrtf(block_sum(ss, scratch) / (float)dim + eps);
    // every thread reads back only what it wrote itself
    for (int d = threadIdx.x; d < dim; d += 256) {
        float u = 0.f;
        for (int s = 0; s < S; ++s) u = fmaf(m.in[s], x[(size_t)s * dim + d], u);
        store_from_float(out + (size_t)i * dim + d, u * r * w[d]);
    }
}

// Rows of up to THREADS * VPT * 4 elements (a multiple of 4) and a fixed number of streams: every
// stream is read once with 16-byte loads, the weighted sum stays in registers.
template <typename T, typename Y, int S, int VPT, int THREADS, int JOIN>
__global__ __launch_bounds__(THREADS) void streams_vec_kernel(
        float* __restrict__ X, const Y* __restrict__ y, int n_parts, size_t part_stride, STMix m,
        const float* __restrict__ w, float eps, const int* __restrict__ rows, T* __restrict__ out, int dim) {
    __shared__ float scratch[16];
    const int i = blockIdx.x;
    float* x = X + (size_t)(rows ? rows[i] : i) * S * dim;
    const int n4 = dim >> 2;
    float4 u[VPT];
    float ss = 0.f;
#pragma unroll
    for (int j = 0; j < VPT; ++j) {
        const int idx = threadIdx.x + j * THREADS;
        u[j] = make_float4(0.f, 0.f, 0.f, 0.f);
        if (idx >= n4) continue;
        float4 old[S];
#pragma unroll
        for (int s = 0; s < S; ++s) old[s] = *(const float4*)(x + (size_t)s * dim + 4 * idx);
        if (JOIN) {
            float4 yv = st_load4(y + (size_t)i * dim + 4 * idx);
            for (int p = 1; p < n_parts; ++p) {
                const float4 a = st_load4(y + p * part_stride + (size_t)i * dim + 4 * idx);
                yv.x += a.x; yv.y += a.y; yv.z += a.z; yv.w += a.w;
            }
#pragma unroll
            for (int t = 0; t < S; ++t) {
                const float o = m.outw[t];
                float4 v = make_float4(o * yv.x, o * yv.y, o * yv.z, o * yv.w);
#pragma unroll
                for (int s = 0; s < S; ++s) v = st_fma(m.mix[s * S + t], old[s], v);
                *(float4*)(x + (size_t)t * dim + 4 * idx) = v;
                if (m.in) u[j] = st_fma(m.in[t], v, u[j]);
            }
        } else {
#pragma unroll
            for (int s = 0; s < S; ++s) u[j] = st_fma(m.in[s], old[s], u[j]);
        }
        ss = fmaf(u[j].x, u[j].x, ss);
        ss = fmaf(u[j].y, u[j].y, ss);
        ss = fmaf(u[j].z, u[j].z, ss);
        ss = fmaf(u[j].w, u[j].w, ss);
    }
    if (!m.in) return;
    const float r = rsqrtf(block_sum(ss, scratch) / (float)dim + eps);
    T* o = out + (size_t)i * dim;
#pragma unroll
    for (int j = 0; j < VPT; ++j) {
        const int idx = threadIdx.x + j * THREADS;
        if (idx < n4) {
            const float4 g = *(const float4*)(w + 4 * idx);
            st_store4(o + 4 * idx, make_float4(u[j].x * r * g.x, u[j].y * r * g.y, u[j].z * r * g.z,
                                               u[j].w * r * g.w));
        }
    }
}

template <typename T, typename Y, int JOIN>
static int st_launch(float* X, const Y* y, int n_parts, STMix m, const float* w, float eps,
                     const int* rows, T* out, int n_rows, int S, int dim, hipStream_t stream) {
    const size_t part_stride = (size_t)n_rows * dim;
    const bool vec = dim % 4 == 0 && dim <= 8192 && S <= 4 && (size_t)X % 16 == 0 && (size_t)y % 16 == 0
        && (size_t)w % 16 == 0 && (size_t)out % 16 == 0;
    if (!vec) {
        streams_kernel<T, Y, JOIN><<<n_rows, 256, 0, stream>>>(X, y, n_parts, part_stride, m, w, eps, rows,
                                                              out, S, dim);
        return GFA_LAUNCH_RESULT();
    }
#define ST_GO(S_, VPT, TH) streams_vec_kernel<T, Y, S_, VPT, TH, JOIN><<<n_rows, TH, 0, stream>>>( \
        X, y, n_parts, part_stride, m, w, eps, rows, out, dim)
#define ST_SIZE(S_) do { if (dim <= 1024) ST_GO(S_, 1, 256); else if (dim <= 4096) ST_GO(S_, 1, 1024); \
                         else ST_GO(S_, 2, 1024); } while (0)
    if (S == 1) ST_SIZE(1);
    else if (S == 2) ST_SIZE(2);
    else if (S == 3) ST_SIZE(3);
    else ST_SIZE(4);
#undef ST_SIZE
#undef ST_GO
    return GFA_LAUNCH_RESULT();
}

extern "C" int gfa_streams_read(const float* X, const float* in, const float* w, float eps,
                                const int* rows, void* out, int out_bf16, int n_rows, int S, int dim,
                                hipStream_t stream) {
    if (n_rows <= 0) return 0;
    if (S < 1 || S > ST_MAX || !in || !w || !out) return (int)hipErrorInvalidValue;
    STMix m{nullptr, nullptr, in};
    float* x = const_cast<float*>(X);                  // a read writes nothing there
    if (out_bf16)
        return st_launch<bf16_t, float, 0>(x, nullptr, 0, m, w, eps, rows, (bf16_t*)out, n_rows, S, dim, stream);
    return st_launch<float, float, 0>(x, nullptr, 0, m, w, eps, rows, (float*)out, n_rows, S, dim, stream);
}

extern "C" int gfa_streams_join(float* X, const void* y, int y_bf16, int n_parts, const float* mix,
                                const float* outw, const float* in, const float* w, float eps, void* out,
                                int out_bf16, int n_rows, int S, int dim, hipStream_t stream) {
    if (n_rows <= 0) return 0;
    if (S < 1 || S > ST_MAX || n_parts < 1 || (y_bf16 && n_parts != 1) || (in && (!w || !out)))
        return (int)hipErrorInvalidValue;
    STMix m{mix, outw, in};
    if (y_bf16) {
        if (out_bf16)
            return st_launch<bf16_t, bf16_t, 1>(X, (const bf16_t*)y, 1, m, w, eps, nullptr, (bf16_t*)out,
                                                n_rows, S, dim, stream);
        return st_launch<float, bf16_t, 1>(X, (const bf16_t*)y, 1, m, w, eps, nullptr, (float*)out, n_rows,
                                           S, dim, stream);
    }
    if (out_bf16)
        return st_launch<bf16_t, float, 1>(X, (const float*)y, n_parts, m, w, eps, nullptr, (bf16_t*)out,
                                           n_rows, S, dim, stream);
    return st_launch<float, float, 1>(X, (const float*)y, n_parts, m, w, eps, nullptr, (float*)out, n_rows, S,
                                      dim, stream);
}
