// Short causal convolutions over time, one per channel, in front of a recurrent cell:
//     y[n, c] = silu(sum_j taps[c, j] x[n - (K - 1) + j, c] + bias[c])         (bias optional)
// over the tokens of n's own sequence; x are C columns of a row of proj (from column `col` on),
// float, and zeros before the sequence's start.  The last K - 1 inputs of every channel are kept
// in the sequence's state slot ([K - 1][C], oldest first, at tail_off) and stand for the tokens
// before the step.  The sum runs over j in order and the bias is added last, in every kernel
// below, so a result does not depend on which one made it.
#include "common.h"

#define SC_MAX_TAPS 16
#define SC_TILE 16                      // tokens a thread of the tiled kernel walks

__device__ __forceinline__ float sc_silu(float z) { return z / (1.f + expf(-z)); }

// One thread per (token, channel); the tails are left as they are.
__global__ __launch_bounds__(256) void short_conv_kernel(
        const float* __restrict__ proj, int row_width, int col, const float* __restrict__ taps,
        const float* __restrict__ bias, int K, int C, const float* __restrict__ state,
        size_t slot_stride, size_t tail_off, const int* __restrict__ tok_seq,
        const int* __restrict__ q_start, const int* __restrict__ slots, float* __restrict__ y,
        int n_tokens) {
    const long long idx = (long long)blockIdx.x * blockDim.x + threadIdx.x;
    if (idx >= (long long)n_tokens * C) return;
    const int n = (int)(idx / C), c = (int)(idx - (long long)n * C);
    const int b = tok_seq[n];
    const int first = q_start[b];
    const float* tail = state + (size_t)slots[b] * slot_stride + tail_off;
    float acc = 0.f;
    for (int j = 0; j < K; ++j) {
        const int src = n - (K - 1) + j;               // a row of this step, if it is the sequence's
        const float x = src >= first ? proj[(size_t)src * row_width + col + c]
                                     : tail[(size_t)(K - 1 + src - first) * C + c];
        acc = fmaf(taps[(size_t)c * K + j], x, acc);
    }
    y[(size_t)n * C + c] = sc_silu(bias ? acc + bias[c] : acc);
}

// Four channels and SC_TILE tokens per thread: every input is read once (16 bytes at a time) and
// slides through registers.  C, col, row_width and the tails' place are multiples of four.
template <int K>
__global__ __launch_bounds__(256) void short_conv_tile_kernel(
        const float* __restrict__ proj, int row_width, int col, const float* __restrict__ taps,
        const float* __restrict__ bias, int C, const float* __restrict__ state, size_t slot_stride,
        size_t tail_off, const int* __restrict__ tok_seq, const int* __restrict__ q_start,
        const int* __restrict__ slots, float* __restrict__ y, int n_tokens) {
    const int c = (blockIdx.x * 256 + threadIdx.x) * 4;
    if (c >= C) return;
    const int n0 = blockIdx.y * SC_TILE, n1 = n0 + SC_TILE < n_tokens ? n0 + SC_TILE : n_tokens;
    float4 w[K], win[K > 1 ? K - 1 : 1];
#pragma unroll
    for (int j = 0; j < K; ++j)
        w[j] = make_float4(taps[(size_t)c * K + j], taps[(size_t)(c + 1) * K + j],
                           taps[(size_t)(c + 2) * K + j], taps[(size_t)(c + 3) * K + j]);
    const float4 bs = bias ? *(const float4*)(bias + c) : make_float4(0.f, 0.f, 0.f, 0.f);
    const float* x = proj + col + c;
    int b = -1;
    for (int n = n0; n < n1; ++n) {
        if (tok_seq[n] != b) {
            b = tok_seq[n];
            const int first = q_start[b];
            const float* tail = state + (size_t)slots[b] * slot_stride + tail_off + c;
#pragma unroll
            for (int i = 0; i < K - 1; ++i) {
                const int src = n - (K - 1) + i;
                win[i] = src >= first ? *(const float4*)(x + (size_t)src * row_width)
                                      : *(const float4*)(tail + (size_t)(K - 1 + src - first) * C);
            }
        }
        const float4 now = *(const float4*)(x + (size_t)n * row_width);
        float4 a = make_float4(0.f, 0.f, 0.f, 0.f);
#pragma unroll
        for (int j = 0; j < K; ++j) {
            const float4 v = j < K - 1 ? win[j < K - 1 ? j : 0] : now;
            a.x = fmaf(w[j].x, v.x, a.x);
            a.y = fmaf(w[j].y, v.y, a.y);
            a.z = fmaf(w[j].z, v.z, a.z);
            a.w = fmaf(w[j].w, v.w, a.w);
        }
#pragma unroll
        for (int i = 0; i + 1 < K - 1; ++i) win[i] = win[i + 1];
        if (K > 1) win[K > 1 ? K - 2 : 0] = now;
        *(float4*)(y + (size_t)n * C + c) = make_float4(sc_silu(a.x + bs.x), sc_silu(a.y + bs.y),
                                                        sc_silu(a.z + bs.z), sc_silu(a.w + bs.w));
    }
}

// Steps of at most one token per sequence: the convolution and the tail's move in one pass.  One
// thread per (sequence, channel).
__global__ __launch_bounds__(256) void short_conv_step_kernel(
        const float* __restrict__ proj, int row_width, int col, const float* __restrict__ taps,
        const float* __restrict__ bias, int K, int C, float* __restrict__ state, size_t slot_stride,
        size_t tail_off, const int* __restrict__ q_start, const int* __restrict__ slots,
        float* __restrict__ y) {
    const int c = blockIdx.x * 256 + threadIdx.x, b = blockIdx.y;
    if (c >= C) return;
    const int n = q_start[b];
    if (q_start[b + 1] <= n) return;
    float* tail = state + (size_t)slots[b] * slot_stride + tail_off + c;
    const float now = proj[(size_t)n * row_width + col + c];
    float acc = 0.f;
    for (int j = 0; j < K - 1; ++j) {
        const float x = tail[(size_t)j * C];
        acc = fmaf(taps[(size_t)c * K + j], x, acc);
        if (j > 0) tail[(size_t)(j - 1) * C] = x;
    }
    if (K > 1) tail[(size_t)(K - 2) * C] = now;
    acc = fmaf(taps[(size_t)c * K + K - 1], now, acc);
    y[(size_t)n * C + c] = sc_silu(bias ? acc + bias[c] : acc);
}

// The tails after the step: the last K - 1 of (old tail, the step's inputs).  One thread per
// (sequence, channel) reads its old entries before it writes.
__global__ __launch_bounds__(256) void conv_tail_kernel(
        const float* __restrict__ proj, int row_width, int col, int K, int C, float* __restrict__ state,
        size_t slot_stride, size_t tail_off, const int* __restrict__ q_start,
        const int* __restrict__ slots, int n_seqs) {
    const long long idx = (long long)blockIdx.x * blockDim.x + threadIdx.x;
    if (idx >= (long long)n_seqs * C) return;
    const int b = (int)(idx / C), c = (int)(idx - (long long)b * C);
    const int first = q_start[b], L = q_start[b + 1] - first;
    float* tail = state + (size_t)slots[b] * slot_stride + tail_off;
    float old[SC_MAX_TAPS];
    for (int i = 0; i < K - 1; ++i) old[i] = tail[(size_t)i * C + c];
    for (int i = 0; i < K - 1; ++i) {
        const int at = L + i;                           // in (old tail, inputs of the step)
        tail[(size_t)i * C + c] = at < K - 1 ? old[at]
                                             : proj[(size_t)(first + at - (K - 1)) * row_width + col + c];
    }
}

extern "C" int gfa_short_conv(const float* proj, int row_width, int col, const float* taps,
                              const float* bias, int K, int C, float* state, size_t slot_stride,
                              size_t tail_off, const int* tok_seq, const int* q_start,
                              const int* slots, float* y, int n_tokens, int n_seqs, int max_q_len,
                              hipStream_t stream) {
    if (n_tokens <= 0 || n_seqs <= 0) return 0;
    if (K < 1 || K > SC_MAX_TAPS || C < 1 || col < 0 || col + C > row_width || n_seqs > 65535)
        return (int)hipErrorInvalidValue;
    if (max_q_len == 1) {
        short_conv_step_kernel<<<dim3((C + 255) / 256, n_seqs), 256, 0, stream>>>(
            proj, row_width, col, taps, bias, K, C, state, slot_stride, tail_off, q_start, slots, y);
        return GFA_LAUNCH_RESULT();
    }
    const int tiles = (n_tokens + SC_TILE - 1) / SC_TILE;
    const bool vec = K <= 4 && C % 4 == 0 && col % 4 == 0 && row_width % 4 == 0 && slot_stride % 4 == 0
        && tail_off % 4 == 0 && (size_t)proj % 16 == 0 && (size_t)state % 16 == 0 && (size_t)y % 16 == 0
        && (size_t)bias % 16 == 0 && tiles <= 65535;
    if (vec) {
        const dim3 grid((C / 4 + 255) / 256, tiles);
#define SC_GO(K_) short_conv_tile_kernel<K_><<<grid, 256, 0, stream>>>( \
        proj, row_width, col, taps, bias, C, state, slot_stride, tail_off, tok_seq, q_start, slots, y, n_tokens)
        if (K == 1) SC_GO(1);
        else if (K == 2) SC_GO(2);
        else if (K == 3) SC_GO(3);
        else SC_GO(4);
#undef SC_GO
    } else {
        const long long units = (long long)n_tokens * C;
        short_conv_kernel<<<(unsigned)((units + 255) / 256), 256, 0, stream>>>(
            proj, row_width, col, taps, bias, K, C, state, slot_stride, tail_off, tok_seq, q_start,
            slots, y, n_tokens);
    }
    if (K > 1) {
        const long long tails = (long long)n_seqs * C;
        conv_tail_kernel<<<(unsigned)((tails + 255) / 256), 256, 0, stream>>>(
            proj, row_width, col, K, C, state, slot_stride, tail_off, q_start, slots, n_seqs);
    }
    return GFA_LAUNCH_RESULT();
}
