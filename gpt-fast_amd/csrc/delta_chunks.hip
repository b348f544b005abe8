// The gated delta rule over many tokens, 64 at a time, in three kernels of which only a small one
// walks the chunks in order.  The cell (gated_delta.hip) per head, with unit k, q (q scaled) and a
// diagonal decay g_t (a number per key channel, or one for the head):
//     S <- g_t S;   u_t = beta_t (v_t - S^T k_t);   S <- S + k_t u_t^T;   o_t = S^T q_t
// With G_t = sum_{r<=t} ln g_r inside a chunk (a vector over the channels), K+ = exp(G) k,
// Q+ = exp(G) q, K- = exp(G_L - G) k (row by row) and, over channels d,
//     A[t][s] = beta_t sum_d k_t k_s exp(G_t - G_s)  (s < t)      P[t][s] = sum_d q_t k_s exp(G_t - G_s)  (s <= t)
// the recurrence written out from the chunk's first state S0 is, with T = (I + A)^-1,
//     W = T diag(beta) K+      U0 = T diag(beta) V      u = U0 - W S0
//     O = (Q+ - P W) S0 + P U0
//     S_L = (diag(exp(G_L)) - K-^T W) S0 + K-^T U0  =  M S0 + B
// 1. chunk kernel (a workgroup per chunk and head, all at once): M, B, Q' = Q+ - P W, P U0;
// 2. state kernel (per head and 16 value columns): S <- M S + B from chunk to chunk, every S0 kept;
// 3. output kernel (per chunk and head): O += Q' S0.
// All products are v_mfma_f32_16x16x4_f32 (lane l supplies A[l % 16][l / 16] and B[l / 16][l % 16] and
// holds C[4 (l / 16) .. + 3][l % 16]).
//
// No exponent above zero: a chunk is four tiles of 16 tokens, and L_t is the sum inside the tile
// (E at its end).  Two tokens of different tiles meet as exp(L_t) k_t times exp(E - L_s) k_s times the
// whole tiles between them, three factors of at most one.  Two tokens of one tile meet as exp(L_t) k_t
// times exp(E - L_s) k_s exp(-E); where a channel's E is below DL_FAR that last factor is too large a
// number, and the tile's 136 pairs are summed one by one with exp(L_t - L_s).  A decay below
// exp(DL_FLOOR) counts as that: what it leaves is below the last digit of what it multiplies.
#include "common.h"

#define DL 64                           // tokens per chunk
#define DL_THREADS 512
#define DL_TILE 272                     // floats of a 16 x 16 tile in shared memory: rows of 17
#define DL_VC 64                        // value columns per pass
#define DL_VS (DL_VC + 4)
#define DL_FLOOR -40.f
#define DL_FAR -60.f
#define DL_MAX_KT 8                     // key channels: up to 16 * this

typedef __attribute__((__vector_size__(4 * sizeof(float)))) float dl_floatx4_t;

struct DLShape {
    int H, G, dk, dv, dvp;              // dvp: dv up to a multiple of 16
    int conv_width, row_width, b_off, a_off;
    const float* decays;                // pre-activations of a decay per channel, [.., H dk], or null: proj's a_off
    int decay_width;
    float q_scale, unit_eps;
    int seg, chunk0;                    // chunks per sequence in this call, and the first one's number
};

__device__ __forceinline__ float dl_softplus(float z) { return z > 20.f ? z : log1pf(expf(z)); }
__device__ __forceinline__ dl_floatx4_t dl_mfma(float a, float b, dl_floatx4_t c) {
    return __builtin_amdgcn_mfma_f32_16x16x4f32(a, b, c, 0, 0, 0);
}
__host__ __device__ inline int dl_tri(int ti, int si) { return ti * (ti + 1) / 2 + si; }

// floats of shared memory of the chunk kernel
static inline int dl_lds_floats(int kt) {
    return 3 * DL * (kt * 16 + 4) + 20 * DL_TILE + 5 * 4 * kt * 16 + DL * DL_VS + DL + 4;
}

template <int KT, bool VEC>
__global__ __launch_bounds__(DL_THREADS) void delta_chunk_kernel(
        const float* __restrict__ conv, const float* __restrict__ proj, const float* __restrict__ A_log,
        const float* __restrict__ dt_bias, const int* __restrict__ q_start, float* __restrict__ wsM,
        float* __restrict__ wsB, float* __restrict__ wsQ, float* __restrict__ out, DLShape s) {
    extern __shared__ __attribute__((aligned(16))) float dl_lds[];
    constexpr int DKP = KT * 16, KS = DKP + 4;
    float* Qs = dl_lds;                          // [DL][KS]  unit q (scaled); then exp(L) q
    float* Ks = Qs + DL * KS;                    // [DL][KS]  unit k; then exp(L) k; then W
    float* Ls = Ks + DL * KS;                    // [DL][KS]  ln g; then L; then exp(E - L) k
    float* At = Ls + DL * KS;                    // [10][16][17]  tiles of A on and below the diagonal; diagonal: then T's
    float* Pt = At + 10 * DL_TILE;               // [10][16][17]
    float* lE = Pt + 10 * DL_TILE;               // [4][DKP]  E of each tile
    float* ex = lE + 4 * DKP;                    // [4][DKP]  exp(E)
    float* inv = ex + 4 * DKP;                   // [4][DKP]  exp(-E)
    float* pre = inv + 4 * DKP;                  // [4][DKP]  decay from the chunk's start to the tile's
    float* suf = pre + 4 * DKP;                  // [4][DKP]  decay from the tile's end to the chunk's
    float* Xv = suf + 4 * DKP;                   // [DL][DL_VS]  beta v, then U0, of the pass's columns
    float* bet = Xv + DL * DL_VS;                // [DL]
    int* far_ = (int*)(bet + DL);                // [4]  the tile's pairs go one by one

    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const int li = lane & 15, lg = lane >> 4;
    const int h = blockIdx.y, b = blockIdx.z, chunk = s.chunk0 + blockIdx.x;
    const int t0 = q_start[b] + chunk * DL, t1 = q_start[b + 1];
    if (t0 >= t1) return;                        // the whole workgroup
    const int Lc = t1 - t0 < DL ? t1 - t0 : DL;
    const size_t slot = ((size_t)b * s.seg + blockIdx.x) * s.H + h;
    const int kvh = h / (s.H / s.G);
    const float rate = expf(A_log[h]);

    {
        // eight threads per token: unit q and k, the decays' logarithms
        const int t = tid >> 3, sub = tid & 7;
        const bool live = t < Lc;
        const size_t row = (size_t)(t0 + (live ? t : 0));
        const float* cq = conv + row * s.conv_width + kvh * s.dk;
        const float* ck = cq + s.G * s.dk;
        const float* z = s.decays ? s.decays + row * s.decay_width + (size_t)h * s.dk : nullptr;
        const float* zb = s.decays ? dt_bias + (size_t)h * s.dk : nullptr;
        const float one_lg = s.decays ? 0.f
            : fmaxf(DL_FLOOR, -rate * dl_softplus(proj[row * s.row_width + s.a_off + h] + dt_bias[h]));
        float sq = 0.f, sk = 0.f;
        if (VEC) {
            constexpr int NV = (DKP / 4 + 7) / 8;
            float4 rq[NV], rk[NV], rz[NV];
            const int n4 = s.dk >> 2;
            const float4 zero = make_float4(0.f, 0.f, 0.f, 0.f);
#pragma unroll
            for (int i = 0; i < NV; ++i) {
                const int j = sub + 8 * i;
                const bool in = live && j < n4;
                rq[i] = in ? *(const float4*)(cq + 4 * j) : zero;
                rk[i] = in ? *(const float4*)(ck + 4 * j) : zero;
                rz[i] = zero;
                if (in && z) {
                    const float4 a = *(const float4*)(z + 4 * j), c = *(const float4*)(zb + 4 * j);
                    rz[i] = make_float4(fmaxf(DL_FLOOR, -rate * dl_softplus(a.x + c.x)),
                                        fmaxf(DL_FLOOR, -rate * dl_softplus(a.y + c.y)),
                                        fmaxf(DL_FLOOR, -rate * dl_softplus(a.z + c.z)),
                                        fmaxf(DL_FLOOR, -rate * dl_softplus(a.w + c.w)));
                } else if (in) {
                    rz[i] = make_float4(one_lg, one_lg, one_lg, one_lg);
                }
                sq += rq[i].x * rq[i].x + rq[i].y * rq[i].y + rq[i].z * rq[i].z + rq[i].w * rq[i].w;
                sk += rk[i].x * rk[i].x + rk[i].y * rk[i].y + rk[i].z * rk[i].z + rk[i].w * rk[i].w;
            }
#pragma unroll
            for (int o = 1; o < 8; o <<= 1) {
                sq += __shfl_xor(sq, o, 64);
                sk += __shfl_xor(sk, o, 64);
            }
            const float fq = rsqrtf(sq + s.unit_eps) * s.q_scale, fk = rsqrtf(sk + s.unit_eps);
#pragma unroll
            for (int i = 0; i < NV; ++i) {
                const int j = sub + 8 * i;
                if (4 * j >= DKP) continue;
                *(float4*)(Qs + t * KS + 4 * j) = make_float4(rq[i].x * fq, rq[i].y * fq, rq[i].z * fq, rq[i].w * fq);
                *(float4*)(Ks + t * KS + 4 * j) = make_float4(rk[i].x * fk, rk[i].y * fk, rk[i].z * fk, rk[i].w * fk);
                *(float4*)(Ls + t * KS + 4 * j) = rz[i];
            }
        } else {
            for (int e = sub; e < s.dk; e += 8) {
                const float qv = live ? cq[e] : 0.f, kv = live ? ck[e] : 0.f;
                sq = fmaf(qv, qv, sq);
                sk = fmaf(kv, kv, sk);
            }
#pragma unroll
            for (int o = 1; o < 8; o <<= 1) {
                sq += __shfl_xor(sq, o, 64);
                sk += __shfl_xor(sk, o, 64);
            }
            const float fq = rsqrtf(sq + s.unit_eps) * s.q_scale, fk = rsqrtf(sk + s.unit_eps);
            for (int e = sub; e < DKP; e += 8) {
                const bool in = live && e < s.dk;
                Qs[t * KS + e] = in ? cq[e] * fq : 0.f;
                Ks[t * KS + e] = in ? ck[e] * fk : 0.f;
                Ls[t * KS + e] = !in ? 0.f : (z ? fmaxf(DL_FLOOR, -rate * dl_softplus(z[e] + zb[e])) : one_lg);
            }
        }
        if (sub == 0) bet[t] = live ? 1.f / (1.f + expf(-proj[row * s.row_width + s.b_off + h])) : 0.f;
        if (tid < 4) far_[tid] = 0;
    }
    __syncthreads();
    for (int e = tid; e < 4 * DKP; e += DL_THREADS) {
        // the sums inside each tile, a channel per thread
        const int j = e / DKP, d = e % DKP;
        float* p = Ls + j * 16 * KS + d;
        float run = 0.f;
#pragma unroll
        for (int t = 0; t < 16; ++t) {
            run += p[t * KS];
            p[t * KS] = run;
        }
        lE[e] = run;
        ex[e] = expf(run);
        inv[e] = expf(-fmaxf(run, DL_FAR));
        if (run < DL_FAR) far_[j] = 1;           // every writer writes the same
    }
    __syncthreads();
    for (int d = tid; d < DKP; d += DL_THREADS) {
        float p = 1.f, q = 1.f;
#pragma unroll
        for (int j = 0; j < 4; ++j) {
            pre[j * DKP + d] = p;
            p *= ex[j * DKP + d];
            suf[(3 - j) * DKP + d] = q;
            q *= ex[(3 - j) * DKP + d];
        }
    }
    for (int j = 0; j < 4; ++j) {
        if (!far_[j] || tid >= 256) continue;
        // pair by pair: thread (t, s) of the tile
        const int t = tid >> 4, u = tid & 15;
        float a = 0.f, p = 0.f;
        if (u <= t) {
            const int rt = (j * 16 + t) * KS, ru = (j * 16 + u) * KS;
            for (int d = 0; d < DKP; ++d) {
                const float w = Ks[ru + d] * expf(Ls[rt + d] - Ls[ru + d]);
                a = fmaf(Ks[rt + d], w, a);
                p = fmaf(Qs[rt + d], w, p);
            }
        }
        At[dl_tri(j, j) * DL_TILE + t * 17 + u] = u < t ? bet[j * 16 + t] * a : 0.f;
        Pt[dl_tri(j, j) * DL_TILE + t * 17 + u] = p;
    }
    __syncthreads();
    for (int e = tid; e < DL * DKP; e += DL_THREADS) {
        const int t = e / DKP, d = e % DKP, at = t * KS + d;
        const float l = Ls[at], k = Ks[at], up = expf(l);
        Qs[at] *= up;
        Ks[at] = k * up;
        Ls[at] = k * expf(lE[(t >> 4) * DKP + d] - l);
    }
    __syncthreads();
    // tile (ti, si) of A or P; between: channel factors of what lies between the two tiles' decays
    auto pair_tile = [&](int ti, int si, bool is_p) {
        dl_floatx4_t acc = {0.f, 0.f, 0.f, 0.f};
        const float* ra = (is_p ? Qs : Ks) + (ti * 16 + li) * KS + lg;
        const float* kb = Ls + (si * 16 + li) * KS + lg;
        const float* f1 = ti == si ? inv + ti * DKP + lg : ex + (si + 1) * DKP + lg;
        const float* f2 = ex + (si + 2 < 4 ? si + 2 : 3) * DKP + lg;
        const int between = ti == si ? 1 : ti - si - 1;
        if (between == 0) {
#pragma unroll 8
            for (int d0 = 0; d0 < DKP; d0 += 4) acc = dl_mfma(ra[d0], kb[d0], acc);
        } else if (between == 1) {
#pragma unroll 8
            for (int d0 = 0; d0 < DKP; d0 += 4) acc = dl_mfma(ra[d0], kb[d0] * f1[d0], acc);
        } else {
#pragma unroll 8
            for (int d0 = 0; d0 < DKP; d0 += 4) acc = dl_mfma(ra[d0], kb[d0] * (f1[d0] * f2[d0]), acc);
        }
        float* dst = (is_p ? Pt : At) + dl_tri(ti, si) * DL_TILE;
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const int t = lg * 4 + r;
            float v = acc[r];
            if (ti == si) v = (is_p ? li <= t : li < t) ? v : 0.f;
            dst[t * 17 + li] = is_p ? v : bet[ti * 16 + t] * v;
        }
    };
    if (!far_[wave >> 1]) pair_tile(wave >> 1, wave >> 1, wave & 1);
    __syncthreads();
    if (wave == 0) {
        // (I + A_jj)^-1 of the four diagonal tiles, a column per lane, in place of A_jj
        float* a = At + dl_tri(lg, lg) * DL_TILE;
        float x[16];
#pragma unroll
        for (int t = 0; t < 16; ++t) {
            float v = t == li ? 1.f : 0.f;
#pragma unroll
            for (int u = 0; u < t; ++u) v = fmaf(-a[t * 17 + u], x[u], v);
            x[t] = v;
        }
#pragma unroll
        for (int t = 0; t < 16; ++t) a[t * 17 + li] = x[t];
    } else {
        for (int i = wave - 1; i < 12; i += 7) {
            const int k = i % 6;                 // (1,0) (2,0) (2,1) (3,0) (3,1) (3,2)
            const int ti = k == 0 ? 1 : (k < 3 ? 2 : 3), si = k - (ti - 1) * ti / 2;
            pair_tile(ti, si, i >= 6);
        }
    }
    __syncthreads();
    // X = T R for 16 columns, in place: block row i is T_ii (R_i - sum_{j<i} A_ij X_j).  A wave owns its
    // columns, so nobody else reads or writes them meanwhile.
    auto solve = [&](float* X, int stride) {
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            dl_floatx4_t acc;
#pragma unroll
            for (int r = 0; r < 4; ++r) acc[r] = X[(i * 16 + lg * 4 + r) * stride + li];
            for (int j = 0; j < i; ++j) {
                const float* a = At + dl_tri(i, j) * DL_TILE + li * 17 + lg;
                const float* x = X + (j * 16 + lg) * stride + li;
#pragma unroll
                for (int k = 0; k < 16; k += 4) acc = dl_mfma(-a[k], x[k * stride], acc);
            }
#pragma unroll
            for (int r = 0; r < 4; ++r) X[(i * 16 + lg * 4 + r) * stride + li] = acc[r];
            const float* a = At + dl_tri(i, i) * DL_TILE + li * 17 + lg;
            const float* x = X + (i * 16 + lg) * stride + li;
            dl_floatx4_t y = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int k = 0; k < 16; k += 4) y = dl_mfma(a[k], x[k * stride], y);
#pragma unroll
            for (int r = 0; r < 4; ++r) X[(i * 16 + lg * 4 + r) * stride + li] = y[r];
        }
    };
    if (wave < KT) {
        float* X = Ks + wave * 16;
#pragma unroll
        for (int i = 0; i < 4; ++i)
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                const int t = i * 16 + lg * 4 + r;
                X[t * KS + li] *= bet[t] * pre[i * DKP + wave * 16 + li];
            }
        solve(X, KS);
    }
    // tile (di, 16 columns of X at `col`) of K-^T X
    auto back_tile = [&](int di, const float* X, int stride) {
        dl_floatx4_t acc = {0.f, 0.f, 0.f, 0.f};
        const float* ka = Ls + lg * KS + di * 16 + li;
        const float* x = X + lg * stride + li;
#pragma unroll
        for (int j = 0; j < 4; ++j) {
            const float f = suf[j * DKP + di * 16 + li];
#pragma unroll
            for (int k = 0; k < 16; k += 4)
                acc = dl_mfma(ka[(j * 16 + k) * KS] * f, x[(j * 16 + k) * stride], acc);
        }
        return acc;
    };
    // tile (ti, 16 columns of X) of P X
    auto forth_tile = [&](int ti, const float* X, int stride) {
        dl_floatx4_t acc = {0.f, 0.f, 0.f, 0.f};
        for (int j = 0; j <= ti; ++j) {
            const float* p = Pt + dl_tri(ti, j) * DL_TILE + li * 17 + lg;
            const float* x = X + (j * 16 + lg) * stride + li;
#pragma unroll
            for (int k = 0; k < 16; k += 4) acc = dl_mfma(p[k], x[k * stride], acc);
        }
        return acc;
    };
    for (int v0 = 0; v0 < s.dv; v0 += DL_VC) {
        const int vt = (s.dv - v0 + 15) / 16 < DL_VC / 16 ? (s.dv - v0 + 15) / 16 : DL_VC / 16;
        for (int e = tid; e < DL * DL_VC; e += DL_THREADS) {
            const int t = e / DL_VC, c = e % DL_VC;
            float v = 0.f;
            if (t < Lc && v0 + c < s.dv)
                v = conv[(size_t)(t0 + t) * s.conv_width + 2 * s.G * s.dk + (size_t)h * s.dv + v0 + c] * bet[t];
            Xv[t * DL_VS + c] = v;
        }
        __syncthreads();
        if (wave < vt) solve(Xv + wave * 16, DL_VS);
        __syncthreads();
        for (int i = wave; i < 4 * vt; i += 8) {
            const int ti = i / vt, ci = i % vt, c = v0 + ci * 16 + li;
            const dl_floatx4_t acc = forth_tile(ti, Xv + ci * 16, DL_VS);
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                const int t = ti * 16 + lg * 4 + r;
                if (t < Lc && c < s.dv) out[(size_t)(t0 + t) * s.H * s.dv + (size_t)h * s.dv + c] = acc[r];
            }
        }
        for (int i = wave; i < KT * vt; i += 8) {
            const int di = i / vt, ci = i % vt;
            const dl_floatx4_t acc = back_tile(di, Xv + ci * 16, DL_VS);
#pragma unroll
            for (int r = 0; r < 4; ++r)
                wsB[(slot * DKP + di * 16 + lg * 4 + r) * s.dvp + v0 + ci * 16 + li] = acc[r];
        }
        __syncthreads();                         // the next pass's columns go to the same place
    }
    // (the barriers above also lie between W's solution and its readers)
    for (int i = wave; i < 4 * KT; i += 8) {
        const int ti = i / KT, ci = i % KT, d = ci * 16 + li;
        const dl_floatx4_t acc = forth_tile(ti, Ks + ci * 16, KS);
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const int t = ti * 16 + lg * 4 + r;
            wsQ[(slot * DL + t) * DKP + d] = Qs[t * KS + d] * pre[ti * DKP + d] - acc[r];
        }
    }
    for (int i = wave; i < KT * KT; i += 8) {
        const int di = i / KT, ci = i % KT, col = ci * 16 + li;
        const dl_floatx4_t acc = back_tile(di, Ks + ci * 16, KS);
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const int d = di * 16 + lg * 4 + r;
            const float whole = d == col ? pre[3 * DKP + d] * ex[3 * DKP + d] : 0.f;
            wsM[(slot * DKP + d) * DKP + col] = whole - acc[r];
        }
    }
}

// S <- M S + B over a sequence's chunks, 16 value columns of one head per workgroup (grid dvp / 16, H,
// sequences).  S lies transposed in shared memory; every chunk's S0 goes to wsS [slot][dvp][DKP].
// Inside a group of 16 key channels lane group lg takes channels 4 lg .. + 3, one per product.
template <int KT>
__global__ __launch_bounds__(256) void delta_state_kernel(
        float* __restrict__ state, size_t slot_stride, const int* __restrict__ q_start,
        const int* __restrict__ slots, const float* __restrict__ wsM, const float* __restrict__ wsB,
        float* __restrict__ wsS, DLShape s) {
    constexpr int DKP = KT * 16, SS = DKP + 4, RT = (KT + 3) / 4;
    __shared__ __attribute__((aligned(16))) float St[16 * SS];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const int li = lane & 15, lg = lane >> 4;
    const int h = blockIdx.y, b = blockIdx.z, col0 = blockIdx.x * 16;
    const int len = q_start[b + 1] - q_start[b];
    int n = (len + DL - 1) / DL - s.chunk0;
    n = n < s.seg ? n : s.seg;
    if (n <= 0) return;                          // the whole workgroup
    float* const S = state + (size_t)slots[b] * slot_stride + (size_t)h * s.dk * s.dv;
    for (int e = tid; e < 16 * DKP; e += 256) {
        const int d = e >> 4, c = e & 15;
        St[c * SS + d] = (d < s.dk && col0 + c < s.dv) ? S[(size_t)d * s.dv + col0 + c] : 0.f;
    }
    float4 m[RT][KT], bias[RT];
    auto fetch = [&](int i) {
        const size_t slot = ((size_t)b * s.seg + i) * s.H + h;
#pragma unroll
        for (int j = 0; j < RT; ++j) {
            const int di = wave + 4 * j;
            if (di >= KT) continue;
#pragma unroll
            for (int k = 0; k < KT; ++k)
                m[j][k] = *(const float4*)(wsM + (slot * DKP + di * 16 + li) * DKP + k * 16 + lg * 4);
            const float* bp = wsB + (slot * DKP + di * 16 + lg * 4) * s.dvp + col0 + li;
            bias[j] = make_float4(bp[0], bp[s.dvp], bp[2 * s.dvp], bp[3 * s.dvp]);
        }
    };
    fetch(0);
    __syncthreads();
    for (int i = 0; i < n; ++i) {
        const size_t slot = ((size_t)b * s.seg + i) * s.H + h;
        for (int e = tid; e < 16 * (DKP / 4); e += 256) {
            const int c = e / (DKP / 4), d4 = e % (DKP / 4);
            *(float4*)(wsS + (slot * s.dvp + col0 + c) * DKP + 4 * d4) = *(const float4*)(St + c * SS + 4 * d4);
        }
        float4 sb[KT];
#pragma unroll
        for (int k = 0; k < KT; ++k) sb[k] = *(const float4*)(St + li * SS + k * 16 + lg * 4);
        dl_floatx4_t acc[RT];
#pragma unroll
        for (int j = 0; j < RT; ++j) {
            if (wave + 4 * j >= KT) continue;
            acc[j] = dl_floatx4_t{bias[j].x, bias[j].y, bias[j].z, bias[j].w};
#pragma unroll
            for (int k = 0; k < KT; ++k) {
                acc[j] = dl_mfma(m[j][k].x, sb[k].x, acc[j]);
                acc[j] = dl_mfma(m[j][k].y, sb[k].y, acc[j]);
                acc[j] = dl_mfma(m[j][k].z, sb[k].z, acc[j]);
                acc[j] = dl_mfma(m[j][k].w, sb[k].w, acc[j]);
            }
        }
        if (i + 1 < n) fetch(i + 1);
        lds_barrier();                           // everyone has read S
#pragma unroll
        for (int j = 0; j < RT; ++j) {
            if (wave + 4 * j >= KT) continue;
            *(float4*)(St + li * SS + (wave + 4 * j) * 16 + lg * 4) =
                make_float4(acc[j][0], acc[j][1], acc[j][2], acc[j][3]);
        }
        lds_barrier();
    }
    for (int e = tid; e < 16 * s.dk; e += 256) {
        const int d = e >> 4, c = e & 15;
        if (col0 + c < s.dv) S[(size_t)d * s.dv + col0 + c] = St[c * SS + d];
    }
}

// out += Q' S0: a workgroup per chunk and head, a wave per tile of 16 tokens.
template <int KT>
__global__ __launch_bounds__(256) void delta_output_kernel(
        const int* __restrict__ q_start, const float* __restrict__ wsQ, const float* __restrict__ wsS,
        float* __restrict__ out, DLShape s) {
    constexpr int DKP = KT * 16;
    const int lane = threadIdx.x & 63, ti = threadIdx.x >> 6;
    const int li = lane & 15, lg = lane >> 4;
    const int h = blockIdx.y, b = blockIdx.z, chunk = s.chunk0 + blockIdx.x;
    const int t0 = q_start[b] + chunk * DL, t1 = q_start[b + 1];
    if (t0 + ti * 16 >= t1) return;              // no barrier follows
    const size_t slot = ((size_t)b * s.seg + blockIdx.x) * s.H + h;
    float4 a[KT];
#pragma unroll
    for (int k = 0; k < KT; ++k) a[k] = *(const float4*)(wsQ + (slot * DL + ti * 16 + li) * DKP + k * 16 + lg * 4);
    for (int c0 = 0; c0 < s.dv; c0 += 16) {
        const float* sp = wsS + (slot * s.dvp + c0 + li) * DKP + lg * 4;
        dl_floatx4_t acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int k = 0; k < KT; ++k) {
            const float4 x = *(const float4*)(sp + k * 16);
            acc = dl_mfma(a[k].x, x.x, acc);
            acc = dl_mfma(a[k].y, x.y, acc);
            acc = dl_mfma(a[k].z, x.z, acc);
            acc = dl_mfma(a[k].w, x.w, acc);
        }
        const int c = c0 + li;
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const int t = t0 + ti * 16 + lg * 4 + r;
            if (t < t1 && c < s.dv) out[(size_t)t * s.H * s.dv + (size_t)h * s.dv + c] += acc[r];
        }
    }
}

static int dl_lds_limit() {
    static int limit = -1;
    if (limit < 0) {
        int dev = 0, v = 0;
        if (hipGetDevice(&dev) != hipSuccess ||
            hipDeviceGetAttribute(&v, hipDeviceAttributeMaxSharedMemoryPerBlock, dev) != hipSuccess)
            v = 64 * 1024;
        limit = v;
    }
    return limit;
}

static int dl_tiles(int dk) {                    // tiles of 16 key channels the kernels are built for
    const int kt = (dk + 15) / 16;
    return kt <= 2 ? 2 : (kt <= 4 ? 4 : (kt <= 6 ? 6 : 8));
}

extern "C" int gfa_delta_chunks_take(int dk, int dv) {
    return dk >= 1 && dv >= 1 && dk <= 16 * DL_MAX_KT
        && dl_lds_floats(dl_tiles(dk)) * (int)sizeof(float) <= dl_lds_limit() ? 1 : 0;
}

// floats of the workspaces per (sequence, chunk, head): M, B, S0, Q'
extern "C" int gfa_delta_chunks_floats(int dk, int dv, int* m, int* b, int* s0, int* q) {
    const int dkp = dl_tiles(dk) * 16, dvp = (dv + 15) / 16 * 16;
    *m = dkp * dkp;
    *b = dkp * dvp;
    *s0 = dkp * dvp;
    *q = DL * dkp;
    return 0;
}

template <int KT>
static int dl_launch(const float* conv, const float* proj, const float* A_log, const float* dt_bias,
                     float* state, size_t slot_stride, const int* q_start, const int* slots, float* out,
                     float* wsM, float* wsB, float* wsS, float* wsQ, int n_seqs, int n_chunks, bool vec,
                     DLShape s, hipStream_t stream) {
    const int bytes = dl_lds_floats(KT) * (int)sizeof(float);
    if (bytes > 64 * 1024) {
        static bool allowed = false;
        if (!allowed) {
            hipError_t e = hipFuncSetAttribute((const void*)delta_chunk_kernel<KT, true>,
                                               hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024);
            if (e == hipSuccess)
                e = hipFuncSetAttribute((const void*)delta_chunk_kernel<KT, false>,
                                        hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024);
            if (e != hipSuccess) return (int)e;
            allowed = true;
        }
    }
    for (s.chunk0 = 0; s.chunk0 < n_chunks; s.chunk0 += s.seg) {
        const int now = n_chunks - s.chunk0 < s.seg ? n_chunks - s.chunk0 : s.seg;
        const dim3 grid(now, s.H, n_seqs);
        if (vec)
            delta_chunk_kernel<KT, true><<<grid, DL_THREADS, bytes, stream>>>(conv, proj, A_log, dt_bias, q_start,
                                                                             wsM, wsB, wsQ, out, s);
        else
            delta_chunk_kernel<KT, false><<<grid, DL_THREADS, bytes, stream>>>(conv, proj, A_log, dt_bias, q_start,
                                                                              wsM, wsB, wsQ, out, s);
        delta_state_kernel<KT><<<dim3(s.dvp / 16, s.H, n_seqs), 256, 0, stream>>>(state, slot_stride, q_start,
                                                                                 slots, wsM, wsB, wsS, s);
        delta_output_kernel<KT><<<grid, 256, 0, stream>>>(q_start, wsQ, wsS, out, s);
    }
    return GFA_LAUNCH_RESULT();
}

// ws*: room for n_seqs * seg * H chunks each; chunks of every sequence are taken `seg` at a time.
extern "C" int gfa_delta_chunks(const float* conv, int conv_width, const float* proj, int row_width, int b_off,
                                int a_off, const float* decays, int decay_width, const float* A_log,
                                const float* dt_bias, float* state, size_t slot_stride, const int* q_start,
                                const int* slots, float* out, float* wsM, float* wsB, float* wsS, float* wsQ,
                                int n_seqs, int max_q_len, int seg, int H, int G, int dk, int dv,
                                float q_scale, float unit_eps, hipStream_t stream) {
    if (n_seqs <= 0 || max_q_len <= 0) return 0;
    if (H < 1 || H > 65535 || G < 1 || H % G || n_seqs > 65535 || seg < 1 || conv_width < 2 * G * dk + H * dv
            || b_off + H > row_width || (!decays && a_off + H > row_width) || (decays && decay_width < H * dk)
            || !gfa_delta_chunks_take(dk, dv))
        return (int)hipErrorInvalidValue;
    DLShape s{H, G, dk, dv, (dv + 15) / 16 * 16, conv_width, row_width, b_off, a_off, decays, decay_width,
              q_scale, unit_eps, seg, 0};
    const int n_chunks = (max_q_len + DL - 1) / DL;
    const bool vec = dk % 4 == 0 && conv_width % 4 == 0 && (size_t)conv % 16 == 0
        && (!decays || (decay_width % 4 == 0 && (size_t)decays % 16 == 0 && (size_t)dt_bias % 16 == 0));
#define DL_GO(KT) return dl_launch<KT>(conv, proj, A_log, dt_bias, state, slot_stride, q_start, slots, out, \
                                       wsM, wsB, wsS, wsQ, n_seqs, n_chunks, vec, s, stream)
    switch (dl_tiles(dk)) {
        case 2: DL_GO(2);
        case 4: DL_GO(4);
        case 6: DL_GO(6);
        default: DL_GO(8);
    }
#undef DL_GO
}
