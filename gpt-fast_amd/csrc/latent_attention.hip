// Attention of many query heads to ONE cached key / value head (latent attention in the latent's
// space: keys of hd = latent + rotated part, values of vd = latent) on the matrix cores,
// bfloat16, over the paged cache:
//     out_h(i) = sum_j softmax_j((q_h(i) . k(j)) scale) v(j) * sigmoid(gate[i, h])     (gate optional)
// over max(0, i - window + 1) <= j <= i (window 0: from 0).
//
// A row is a (token, head) pair, sixteen rows a tile; both products are formed transposed, as in
// scored_attention.hip (S^T = K Q^T, O^T = V^T P^T), so operands lie in the order the cache has.
// What is different here is that the heads share their keys: a block of 32 keys and their values
// (up to 36 + 32 KB) is copied once into shared memory by the whole workgroup (global_load_lds,
// 16 bytes a lane, no registers between) and read from there by every tile.  Single-token steps
// cut the keys into parts over workgroups; a second kernel adds the parts up.
//
// The buffers are LDS objects of their own, named statically: the compiler then knows that a
// copy into one of them does not change what is read from another.
#include "common.h"

typedef __attribute__((__vector_size__(8 * sizeof(__bf16)))) __bf16 la_bf16x8_t;
typedef __attribute__((__vector_size__(4 * sizeof(float)))) float la_floatx4_t;
union LAFrag {
    uint4 u;
    bf16_t e[8];
    la_bf16x8_t v;
};

// a row's reference maximum is raised only when a block exceeds it by 2^LA_SLACK: the output is
// then rescaled rarely, and sums and the bfloat16 weights hold such values at full precision
#define LA_SLACK 8.0f

struct LAShape {
    int H, hd, vd;
    long long q_tok, q_head, o_tok, o_head;      // strides in elements
    int table_stride, window;
    float scale_log2;
    const float* gate;                           // a row of pre-activations per token, or null
    long long gate_tok;
};

__device__ __forceinline__ float la_max_lane_groups(float v) {
    v = fmaxf(v, __shfl_xor(v, 16, GFA_WAVE));
    return fmaxf(v, __shfl_xor(v, 32, GFA_WAVE));
}
__device__ __forceinline__ float la_sum_lane_groups(float v) {
    v += __shfl_xor(v, 16, GFA_WAVE);
    return v + __shfl_xor(v, 32, GFA_WAVE);
}

// The workgroup's NT threads copy block `bi` of a sequence: its 32 keys (64 hd bytes, in one
// piece) and its values (vd / 16 pieces of 1 KB).
template <int NT, int DK, int DVT>
__device__ __forceinline__ void la_copy(const bf16_t* __restrict__ k_pages, const bf16_t* __restrict__ v_pages,
                                        int page, int bi, int hd, int vd, char* kbuf, char* vbuf) {
    const int tid = threadIdx.x, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const char* ks = (const char*)(k_pages + cache_region(page, 0, 1, hd)) + (size_t)(bi & 1) * 64 * hd;
    const char* vs = (const char*)(v_pages + cache_region(page, 0, 1, vd)) + (size_t)(bi & 1) * 1024;
#pragma unroll
    for (int i = 0; i < (DK * 128 + NT - 1) / NT; ++i) {
        const int u = tid + i * NT;
        if (u < 4 * hd)
            __builtin_amdgcn_global_load_lds((const __attribute__((address_space(1))) void*)(ks + (size_t)u * 16),
                                             (__attribute__((address_space(3))) void*)(kbuf + wave * 1024 + i * NT * 16),
                                             16, 0, 0);
    }
#pragma unroll
    for (int i = 0; i < (DVT * 64 + NT - 1) / NT; ++i) {
        const int u = tid + i * NT;
        if (u < 4 * vd)
            __builtin_amdgcn_global_load_lds(
                (const __attribute__((address_space(1))) void*)(vs + (size_t)(u >> 6) * 2048 + (u & 63) * 16),
                (__attribute__((address_space(3))) void*)(vbuf + wave * 1024 + i * NT * 16), 16, 0, 0);
    }
}

// This thread's copies have arrived; values of keys beyond `last` (whatever the pool held there)
// become zero, by the thread that copied them, so that weight 0 times them is 0.  16-byte piece
// u of a block's values holds keys 8 (u / 16 % 4) .. + 7.
template <int NT, int DVT>
__device__ __forceinline__ void la_landed(int bi, int last, int vd, char* vbuf) {
    asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
    const int ok = last - bi * 32;                     // keys 0 .. ok of the block count
    if (ok >= 31) return;
#pragma unroll
    for (int i = 0; i < (DVT * 64 + NT - 1) / NT; ++i) {
        const int u = threadIdx.x + i * NT, first = ((u >> 4) & 3) * 8;
        if (u < 4 * vd && first + 7 > ok) {
            LAFrag f;
            f.u = *(const uint4*)(vbuf + (size_t)u * 16);
#pragma unroll
            for (int e = 0; e < 8; ++e)
                if (first + e > ok) f.e[e] = 0;
            *(uint4*)(vbuf + (size_t)u * 16) = f.u;
        }
    }
}

// One tile of rows: its queries, running maximum and sum, and O^T.
template <int DK, int DVT>
struct LATile {
    LAFrag qf[DK];
    la_floatx4_t o[DVT];
    float m, l;
    int pos, lo;                                       // the row's position (-1: no row), its first key

    __device__ __forceinline__ void start(const bf16_t* __restrict__ qrow, bool valid, int hd) {
        const int lg = (threadIdx.x & 63) >> 4;
#pragma unroll
        for (int kk = 0; kk < DK; ++kk) {
            const int d = kk * 32 + lg * 8;
            qf[kk].u = make_uint4(0, 0, 0, 0);
            if (valid && d < hd) qf[kk].u = *(const uint4*)(qrow + d);
        }
#pragma unroll
        for (int dt = 0; dt < DVT; ++dt) o[dt] = la_floatx4_t{0.f, 0.f, 0.f, 0.f};
        m = -INFINITY;
        l = 0.f;
    }

    // FULL: hd and vd are exactly the sizes of the template
    template <bool FULL>
    __device__ __forceinline__ void block(int bi, const char* kt, const char* vt, int hd, int vd, float scale_log2) {
        const int lane = threadIdx.x & 63, li = lane & 15, lg = lane >> 4;
        const int chunks = hd >> 3, vtiles = vd >> 4;
        la_floatx4_t s0 = {0.f, 0.f, 0.f, 0.f}, s1 = {0.f, 0.f, 0.f, 0.f};
        const char* kl = kt + lg * 512 + li * 16;
#pragma unroll
        for (int kk = 0; kk < DK; ++kk) {
            // beyond the keys' size q is zero: any chunk that holds numbers will do
            const char* src = (FULL || kk * 4 + lg < chunks) ? kl + kk * 2048 : kt + li * 16;
            LAFrag k0, k1;
            k0.u = *(const uint4*)src;
            k1.u = *(const uint4*)(src + 256);
            s0 = __builtin_amdgcn_mfma_f32_16x16x32_bf16(k0.v, qf[kk].v, s0, 0, 0, 0);
            s1 = __builtin_amdgcn_mfma_f32_16x16x32_bf16(k1.v, qf[kk].v, s1, 0, 0, 0);
        }
        float sv[8] = {s0[0], s0[1], s0[2], s0[3], s1[0], s1[1], s1[2], s1[3]};
        const int key0 = bi * 32 + lg * 8;
        float mx = -INFINITY;
#pragma unroll
        for (int e = 0; e < 8; ++e) {
            const int j = key0 + e;
            sv[e] = (j <= pos && j >= lo) ? sv[e] * scale_log2 : -INFINITY;
            mx = fmaxf(mx, sv[e]);
        }
        mx = la_max_lane_groups(mx);
        const bool raise = mx > m + LA_SLACK || m == -INFINITY;
        if (__ballot(raise)) {
            const float to = raise ? fmaxf(m, mx) : m;
            const float f = to == m ? 1.f : exp2f(m - to);      // m = -inf: 0
            l *= f;
            m = to;
#pragma unroll
            for (int dt = 0; dt < DVT; ++dt) o[dt] *= f;
        }
        const float ref = m == -INFINITY ? 0.f : m;
        LAFrag pf;
#pragma unroll
        for (int e = 0; e < 8; ++e) {
            const float p = exp2f(sv[e] - ref);
            l += p;
            pf.e[e] = float_to_bf16(p);
        }
        const char* vl = vt + lane * 16;
#pragma unroll
        for (int dt = 0; dt < DVT; ++dt) {
            LAFrag vf;
            vf.u = *(const uint4*)(vl + (FULL || dt < vtiles ? dt : 0) * 1024);
            o[dt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf.v, pf.v, o[dt], 0, 0, 0);
        }
    }
};

__device__ __forceinline__ void la_store4(bf16_t* dst, float a, float b, float c, float d) {
    uint32_t* w = (uint32_t*)dst;
    w[0] = (uint32_t)float_to_bf16(a) | ((uint32_t)float_to_bf16(b) << 16);
    w[1] = (uint32_t)float_to_bf16(c) | ((uint32_t)float_to_bf16(d) << 16);
}

// Prompts and portions: eight waves, a tile of sixteen rows each; one workgroup per 128 rows of a
// sequence, those with the most keys first.  The copies of the next block run while this one is
// multiplied; one barrier a block.  grid (tiles of 128 rows, 1, sequences).
#define LA_WAVES 8
template <int DK, int DVT, bool FULL>
__global__ __launch_bounds__(LA_WAVES * 64, 2) void latent_prompt_kernel(
        const bf16_t* __restrict__ q, const bf16_t* __restrict__ k_pages, const bf16_t* __restrict__ v_pages,
        const int* __restrict__ q_start, const int* __restrict__ start_pos, const int* __restrict__ table,
        bf16_t* __restrict__ out, LAShape s) {
    constexpr int NT = LA_WAVES * 64;
    __shared__ __attribute__((aligned(16))) char kb0[DK * 2048];
    __shared__ __attribute__((aligned(16))) char kb1[DK * 2048];
    __shared__ __attribute__((aligned(16))) char vb0[DVT * 1024];
    __shared__ __attribute__((aligned(16))) char vb1[DVT * 1024];
    const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
    const int li = lane & 15, lg = lane >> 4;
    const int seq = blockIdx.z;
    const int q0 = q_start[seq], rows_total = (q_start[seq + 1] - q0) * s.H;
    const int wg_row0 = (gridDim.x - 1 - blockIdx.x) * (LA_WAVES * 16);
    if (wg_row0 >= rows_total) return;                 // the whole workgroup
    const int spos = start_pos[seq];
    const int* pages = table + (size_t)seq * s.table_stride;
    auto first_seen = [&](int pos) { return (s.window > 0 && pos - s.window + 1 > 0) ? pos - s.window + 1 : 0; };

    const int row0 = wg_row0 + wave * 16, row = row0 + li;
    const bool valid = row < rows_total;
    const int tok = valid ? row / s.H : 0, head = valid ? row - tok * s.H : 0;
    LATile<DK, DVT> t;
    t.start(q + (size_t)(q0 + tok) * s.q_tok + (size_t)head * s.q_head, valid, s.hd);
    t.pos = valid ? spos + tok : -1;
    t.lo = first_seen(spos + tok);
    // the blocks of the workgroup and of this wave (none: hi < lo)
    const int wg_end = wg_row0 + LA_WAVES * 16 < rows_total ? wg_row0 + LA_WAVES * 16 : rows_total;
    const int wg_last = spos + (wg_end - 1) / s.H;
    const int b_lo = first_seen(spos + wg_row0 / s.H) >> 5, b_hi = wg_last >> 5;
    const int w_end = row0 + 16 < rows_total ? row0 + 16 : rows_total;
    const int w_lo = row0 < rows_total ? first_seen(spos + row0 / s.H) >> 5 : 0;
    const int w_hi = row0 < rows_total ? (spos + (w_end - 1) / s.H) >> 5 : -1;

    la_copy<NT, DK, DVT>(k_pages, v_pages, pages[b_lo >> 1], b_lo, s.hd, s.vd, kb0, vb0);
#define LA_STEP(B, K, V, KN, VN)                                                                        \
    {                                                                                                   \
        la_landed<NT, DVT>(B, wg_last, s.vd, V);                                                        \
        __syncthreads();               /* block B is whole, and nobody reads the other buffers any more */ \
        if ((B) + 1 <= b_hi)                                                                            \
            la_copy<NT, DK, DVT>(k_pages, v_pages, pages[((B) + 1) >> 1], (B) + 1, s.hd, s.vd, KN, VN); \
        if ((B) >= w_lo && (B) <= w_hi) t.template block<FULL>(B, K, V, s.hd, s.vd, s.scale_log2);      \
    }
    for (int b = b_lo; b <= b_hi; b += 2) {
        LA_STEP(b, kb0, vb0, kb1, vb1)
        if (b + 1 <= b_hi) LA_STEP(b + 1, kb1, vb1, kb0, vb0)
    }
#undef LA_STEP
    const float l = la_sum_lane_groups(t.l);
    if (!valid) return;
    float inv = l > 0.f ? 1.f / l : 0.f;
    if (s.gate) inv /= 1.f + expf(-s.gate[(size_t)(q0 + tok) * s.gate_tok + head]);
    bf16_t* orow = out + (size_t)(q0 + tok) * s.o_tok + (size_t)head * s.o_head;
#pragma unroll
    for (int dt = 0; dt < DVT; ++dt)
        if (FULL || dt * 16 < s.vd)
            la_store4(orow + dt * 16 + lg * 4, t.o[dt][0] * inv, t.o[dt][1] * inv, t.o[dt][2] * inv, t.o[dt][3] * inv);
}

// Steps of at most one token per sequence: four waves for up to four tiles (64 heads) of one
// sequence and one of `parts` equal parts of its key blocks, two blocks at a time in shared
// memory.  With two tiles a wave takes one tile and one of the two blocks, with four a tile and
// both blocks, with one tile two waves multiply.  What the waves of a tile have is added up
// through shared memory.  parts 1: the result; else per (sequence, head, part) the maximum (in
// units of log 2), the sum and the unscaled O, which latent_parts_kernel adds up.
// grid (parts, groups of 64 heads, sequences).
template <int DK, int DVT, bool FULL>
__global__ __launch_bounds__(256, 1) void latent_step_kernel(
        const bf16_t* __restrict__ q, const bf16_t* __restrict__ k_pages, const bf16_t* __restrict__ v_pages,
        const int* __restrict__ q_start, const int* __restrict__ start_pos, const int* __restrict__ table,
        bf16_t* __restrict__ out, float* __restrict__ part_ml, float* __restrict__ part_o, int parts, LAShape s) {
    constexpr int NT = 256;
    __shared__ __attribute__((aligned(16))) char kb0[DK * 2048];
    __shared__ __attribute__((aligned(16))) char kb1[DK * 2048];
    __shared__ __attribute__((aligned(16))) char vb0[DVT * 1024];
    __shared__ __attribute__((aligned(16))) char vb1[DVT * 1024];
    static_assert(DK * 2048 >= DVT * 1024 + 128, "a tile's result fits a block of keys");
    const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
    const int li = lane & 15, lg = lane >> 4;
    const int seq = blockIdx.z, part = blockIdx.x;
    const int q0 = q_start[seq];
    if (q_start[seq + 1] <= q0) return;                // the whole workgroup
    const int pos = start_pos[seq];
    const int* pages = table + (size_t)seq * s.table_stride;
    const int h0 = blockIdx.y * 64, heads = s.H - h0 < 64 ? s.H - h0 : 64;
    const int tiles = heads > 32 ? 4 : (heads > 16 ? 2 : 1);
    const int tile = wave & (tiles - 1), share = wave / tiles;      // share: which of the two blocks
    const int head = h0 + tile * 16 + li;
    const bool valid = head < s.H;
    const int lo = (s.window > 0 && pos - s.window + 1 > 0) ? pos - s.window + 1 : 0;
    const int b_lo = lo >> 5, n_blocks = (pos >> 5) - b_lo + 1;
    const int per = (n_blocks + parts - 1) / parts;
    const int b0 = b_lo + part * per, b1 = b0 + per < b_lo + n_blocks ? b0 + per : b_lo + n_blocks;

    LATile<DK, DVT> t;
    t.start(q + (size_t)q0 * s.q_tok + (size_t)(valid ? head : 0) * s.q_head, valid, s.hd);
    t.pos = valid ? pos : -1;
    t.lo = lo;
    for (int b = b0; b < b1; b += 2) {
        const bool two = b + 1 < b1;
        if (b > b0) __syncthreads();                   // the blocks before are done with
        la_copy<NT, DK, DVT>(k_pages, v_pages, pages[b >> 1], b, s.hd, s.vd, kb0, vb0);
        if (two) la_copy<NT, DK, DVT>(k_pages, v_pages, pages[(b + 1) >> 1], b + 1, s.hd, s.vd, kb1, vb1);
        la_landed<NT, DVT>(b, pos, s.vd, vb0);
        if (two) la_landed<NT, DVT>(b + 1, pos, s.vd, vb1);
        __syncthreads();
        if (share == 0) t.template block<FULL>(b, kb0, vb0, s.hd, s.vd, s.scale_log2);
        if (two && share == (tiles == 4 ? 0 : 1)) t.template block<FULL>(b + 1, kb1, vb1, s.hd, s.vd, s.scale_log2);
    }
    float l = la_sum_lane_groups(t.l);
    if (tiles < 4) {
        // the second wave of a tile hands over; rows [16][vd] behind sixteen maxima and sums
        __syncthreads();
        float* box = (float*)(tile == 0 ? kb0 : kb1);
        if (share == 1) {
            if (lg == 0) {
                box[li] = t.m;
                box[16 + li] = l;
            }
#pragma unroll
            for (int dt = 0; dt < DVT; ++dt)
                if (FULL || dt * 16 < s.vd)
                    *(la_floatx4_t*)(box + 32 + li * s.vd + dt * 16 + lg * 4) = t.o[dt];
        }
        __syncthreads();
        if (share != 0) return;
        const float m2 = box[li], l2 = box[16 + li];
        const float M = fmaxf(t.m, m2);
        const float f1 = t.m == -INFINITY ? 0.f : exp2f(t.m - M), f2 = m2 == -INFINITY ? 0.f : exp2f(m2 - M);
        l = l * f1 + l2 * f2;
        t.m = M;
#pragma unroll
        for (int dt = 0; dt < DVT; ++dt)
            if (FULL || dt * 16 < s.vd) {
                const la_floatx4_t o2 = *(const la_floatx4_t*)(box + 32 + li * s.vd + dt * 16 + lg * 4);
#pragma unroll
                for (int j = 0; j < 4; ++j) t.o[dt][j] = t.o[dt][j] * f1 + o2[j] * f2;
            }
    }
    if (!valid) return;
    if (parts > 1) {
        const size_t at = ((size_t)seq * s.H + head) * parts + part;
        if (lg == 0) {
            part_ml[2 * at] = t.m;
            part_ml[2 * at + 1] = l;
        }
        if (t.m == -INFINITY) return;                  // a part without keys: its O is not read
#pragma unroll
        for (int dt = 0; dt < DVT; ++dt)
            if (FULL || dt * 16 < s.vd)
                *(la_floatx4_t*)(part_o + at * s.vd + dt * 16 + lg * 4) = t.o[dt];
        return;
    }
    float inv = l > 0.f ? 1.f / l : 0.f;
    if (s.gate) inv /= 1.f + expf(-s.gate[(size_t)q0 * s.gate_tok + head]);
    bf16_t* orow = out + (size_t)q0 * s.o_tok + (size_t)head * s.o_head;
#pragma unroll
    for (int dt = 0; dt < DVT; ++dt)
        if (FULL || dt * 16 < s.vd)
            la_store4(orow + dt * 16 + lg * 4, t.o[dt][0] * inv, t.o[dt][1] * inv, t.o[dt][2] * inv, t.o[dt][3] * inv);
}

// The parts of a head's keys added up in order; grid (heads, sequences), four values a thread.
__global__ __launch_bounds__(128) void latent_parts_kernel(
        const float* __restrict__ part_ml, const float* __restrict__ part_o, int parts,
        const int* __restrict__ q_start, bf16_t* __restrict__ out, LAShape s) {
    const int head = blockIdx.x, seq = blockIdx.y;
    const int q0 = q_start[seq];
    if (q_start[seq + 1] <= q0) return;
    const size_t at = ((size_t)seq * s.H + head) * parts;
    float M = -INFINITY;
    for (int p = 0; p < parts; ++p) M = fmaxf(M, part_ml[2 * (at + p)]);
    const int d = threadIdx.x * 4;
    float l = 0.f, a0 = 0.f, a1 = 0.f, a2 = 0.f, a3 = 0.f;
    for (int p = 0; p < parts; ++p) {
        const float m = part_ml[2 * (at + p)];
        if (m == -INFINITY) continue;
        const float f = exp2f(m - M);
        l = fmaf(part_ml[2 * (at + p) + 1], f, l);
        if (d < s.vd) {
            const float4 o = *(const float4*)(part_o + (at + p) * s.vd + d);
            a0 = fmaf(o.x, f, a0);
            a1 = fmaf(o.y, f, a1);
            a2 = fmaf(o.z, f, a2);
            a3 = fmaf(o.w, f, a3);
        }
    }
    if (d >= s.vd) return;
    float inv = l > 0.f ? 1.f / l : 0.f;
    if (s.gate) inv /= 1.f + expf(-s.gate[(size_t)q0 * s.gate_tok + head]);
    la_store4(out + (size_t)q0 * s.o_tok + (size_t)head * s.o_head + d, a0 * inv, a1 * inv, a2 * inv, a3 * inv);
}

// 1 if these kernels take the sizes (bfloat16, one kv head)
extern "C" int gfa_latent_attention_takes(int H, int hd, int vd) {
    return H >= 1 && hd >= 8 && hd % 8 == 0 && hd <= 576 && vd >= 16 && vd % 16 == 0 && vd <= 512 ? 1 : 0;
}

extern "C" int gfa_latent_attention(const void* q, const void* k_pages, const void* v_pages, const int* q_start,
                                    const int* start_pos, const int* table, int table_stride, void* out,
                                    float* part_ml, float* part_o, int parts, int n_seqs, int max_q_len, int H,
                                    int hd, int vd, long long q_tok, long long q_head, long long o_tok,
                                    long long o_head, float scale, int window, const float* gate,
                                    long long gate_tok, hipStream_t stream) {
    if (n_seqs <= 0 || max_q_len <= 0) return 0;
    if (!gfa_latent_attention_takes(H, hd, vd) || n_seqs > 65535 || q_tok % 8 || q_head % 8 || o_tok % 2 || o_head % 2
            || parts < 1 || parts > 65535 || (parts > 1 && (max_q_len != 1 || !part_ml || !part_o)))
        return (int)hipErrorInvalidValue;
    LAShape s{H, hd, vd, q_tok, q_head, o_tok, o_head, table_stride, window, scale * 1.4426950408889634f, gate, gate_tok};
    const dim3 step_grid(parts, (H + 63) / 64, n_seqs);
    const dim3 prompt_grid((unsigned)(((long long)max_q_len * H + LA_WAVES * 16 - 1) / (LA_WAVES * 16)), 1, n_seqs);
#define LA_GO(DK, DVT, FULL) do {                                                                          \
        if (max_q_len == 1)                                                                                \
            latent_step_kernel<DK, DVT, FULL><<<step_grid, 256, 0, stream>>>(                              \
                (const bf16_t*)q, (const bf16_t*)k_pages, (const bf16_t*)v_pages, q_start, start_pos, table, \
                (bf16_t*)out, part_ml, part_o, parts, s);                                                  \
        else                                                                                               \
            latent_prompt_kernel<DK, DVT, FULL><<<prompt_grid, LA_WAVES * 64, 0, stream>>>(                \
                (const bf16_t*)q, (const bf16_t*)k_pages, (const bf16_t*)v_pages, q_start, start_pos, table, \
                (bf16_t*)out, s);                                                                          \
    } while (0)
    if (hd == 576 && vd == 512) LA_GO(18, 32, true);
    else if (hd <= 192 && vd <= 128) LA_GO(6, 8, false);
    else if (hd <= 320 && vd <= 256) LA_GO(10, 16, false);
    else LA_GO(18, 32, false);
#undef LA_GO
    if (parts > 1)
        latent_parts_kernel<<<dim3(H, n_seqs), 128, 0, stream>>>(part_ml, part_o, parts, q_start, (bf16_t*)out, s);
    return GFA_LAUNCH_RESULT();
}
