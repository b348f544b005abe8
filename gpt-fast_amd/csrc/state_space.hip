// State-space cell with a decay per token (state-space duality, the cell of Mamba-2): per
// sequence and head a float state S [N, dv], zero at the sequence's start and kept in the
// cache's state slots:
//     dt = softplus(dt' + dt_bias_h)           a = exp(-exp(A_log_h) dt)
//     S <- a S + dt B x^T                      y = S^T C + D_h x
// x (H heads of dv), B and C (G groups of N) are the rows that come out of the short convolution,
// side by side [x | B | C]; head h uses group h / (H / G); dt' lies in the projection's rows.
// Everything here is float arithmetic.  One slot's state: S [H][N][dv], then the convolution's
// tails (short_conv.hip).
#include "common.h"

#define SS_THREADS 256
#define SS_COLS 32                      // columns of S (elements of x) per workgroup
#define SS_GROUPS (SS_THREADS / SS_COLS)

struct SSShape {
    int H, G, N, dv;
    int conv_width;                     // floats per row of [x | B | C]
    int row_width, dt_off;              // floats per row of proj, column of the step sizes
};

__device__ __forceinline__ float ss_softplus(float z) { return z > 20.f ? z : log1pf(expf(z)); }

// Token by token.  grid (dv / SS_COLS, H, sequences).  Thread (c, g) = (tid % 32, tid / 32) holds
// rows g, g + 8, ... of column c of S in registers.  B, C and the exchange buffer alternate
// between two copies, so a token costs two barriers; the next token's values are fetched
// meanwhile.
template <int RPT>
__global__ __launch_bounds__(SS_THREADS) void state_space_scan_kernel(
        const float* __restrict__ conv, const float* __restrict__ proj,
        const float* __restrict__ A_log, const float* __restrict__ dt_bias,
        const float* __restrict__ skip, float* __restrict__ state, size_t slot_stride,
        const int* __restrict__ q_start, const int* __restrict__ slots, float* __restrict__ out,
        SSShape s) {
    __shared__ float bs[2][RPT * SS_GROUPS], cs[2][RPT * SS_GROUPS];
    __shared__ float red[2][SS_GROUPS][SS_COLS];
    const int tid = threadIdx.x, c = tid % SS_COLS, g = tid / SS_COLS;
    const int col = blockIdx.x * SS_COLS + c;
    const int h = blockIdx.y, b = blockIdx.z;
    const int grp = h / (s.H / s.G), inner = s.H * s.dv;
    const int t0 = q_start[b], t1 = q_start[b + 1];
    if (t0 >= t1) return;
    float* const S = state + (size_t)slots[b] * slot_stride + (size_t)h * s.N * s.dv;
    const bool col_ok = col < s.dv;
    const int b_col = inner + grp * s.N, c_col = inner + s.G * s.N + grp * s.N, x_col = h * s.dv + col;
    constexpr int EPT = (RPT * SS_GROUPS + SS_THREADS - 1) / SS_THREADS;    // elements of B a thread fetches

    float nb[EPT], nc[EPT], nx = 0.f, nd = 0.f;
    auto fetch = [&](int t) {
        const float* cr = conv + (size_t)t * s.conv_width;
#pragma unroll
        for (int i = 0; i < EPT; ++i) {
            const int e = tid + i * SS_THREADS;
            nb[i] = e < s.N ? cr[b_col + e] : 0.f;
            nc[i] = e < s.N ? cr[c_col + e] : 0.f;
        }
        nx = col_ok ? cr[x_col] : 0.f;
        nd = proj[(size_t)t * s.row_width + s.dt_off + h];
    };
    fetch(t0);
    float Sreg[RPT];
#pragma unroll
    for (int r = 0; r < RPT; ++r) {
        const int row = g + r * SS_GROUPS;
        Sreg[r] = (col_ok && row < s.N) ? S[(size_t)row * s.dv + col] : 0.f;
    }
    const float rate = expf(A_log[h]), bias = dt_bias[h], Dh = skip[h];
    for (int t = t0; t < t1; ++t) {
        const int p = (t - t0) & 1;
#pragma unroll
        for (int i = 0; i < EPT; ++i) {
            const int e = tid + i * SS_THREADS;
            if (e < RPT * SS_GROUPS) {
                bs[p][e] = nb[i];
                cs[p][e] = nc[i];
            }
        }
        const float x = nx;
        const float dt = ss_softplus(nd + bias);
        const float a = expf(-rate * dt), dx = dt * x;
        if (t + 1 < t1) fetch(t + 1);
        __syncthreads();
        float part = 0.f;
#pragma unroll
        for (int r = 0; r < RPT; ++r) {
            const int e = g + r * SS_GROUPS;
            Sreg[r] = fmaf(a, Sreg[r], bs[p][e] * dx);
            part = fmaf(Sreg[r], cs[p][e], part);
        }
        red[p][g][c] = part;
        __syncthreads();
        if (g == 0 && col_ok) {
            float y = 0.f;
#pragma unroll
            for (int r = 0; r < SS_GROUPS; ++r) y += red[p][r][c];
            out[(size_t)t * inner + x_col] = fmaf(Dh, x, y);
        }
    }
#pragma unroll
    for (int r = 0; r < RPT; ++r) {
        const int row = g + r * SS_GROUPS;
        if (col_ok && row < s.N) S[(size_t)row * s.dv + col] = Sreg[r];
    }
}

static bool ss_fits(const SSShape& s, int n_seqs) {
    return s.N >= 1 && s.N <= 64 * SS_GROUPS && s.dv >= 1 && s.H >= 1 && s.H <= 65535 && s.G >= 1
        && s.H % s.G == 0 && n_seqs <= 65535 && s.conv_width >= s.H * s.dv + 2 * s.G * s.N
        && s.dt_off >= 0 && s.dt_off + s.H <= s.row_width;
}

extern "C" int gfa_state_space_scan(const float* conv, int conv_width, const float* proj, int row_width,
                                    int dt_off, const float* A_log, const float* dt_bias,
                                    const float* skip, float* state, size_t slot_stride,
                                    const int* q_start, const int* slots, float* out, int n_seqs, int H,
                                    int G, int N, int dv, hipStream_t stream) {
    if (n_seqs <= 0) return 0;
    SSShape s{H, G, N, dv, conv_width, row_width, dt_off};
    if (!ss_fits(s, n_seqs)) return (int)hipErrorInvalidValue;
    dim3 grid((dv + SS_COLS - 1) / SS_COLS, H, n_seqs);
    const int rpt = (N + SS_GROUPS - 1) / SS_GROUPS;
#define SS_LAUNCH(R) state_space_scan_kernel<R><<<grid, SS_THREADS, 0, stream>>>( \
        conv, proj, A_log, dt_bias, skip, state, slot_stride, q_start, slots, out, s)
    if (rpt <= 4) SS_LAUNCH(4);
    else if (rpt <= 8) SS_LAUNCH(8);
    else if (rpt <= 16) SS_LAUNCH(16);
    else if (rpt <= 32) SS_LAUNCH(32);
    else SS_LAUNCH(64);
#undef SS_LAUNCH
    return GFA_LAUNCH_RESULT();
}

// --------------------------------------------------------------------------------------
// The same cell for runs of many tokens, a chunk of SC_L (32 or 64) tokens at a time.  With S0 the
// state at the chunk's start, t, s = 0, 1, ... the chunk's tokens, L_t = sum_{r<=t} ln a_r and
// e(t, s) = exp(L_t - L_s) <= 1 for s <= t (L in double: one fast decay must not cost the slow ones
// behind it their digits), the recurrence written out is
//     P[t][s] = (C_t . B_s) e(t, s) dt_s  for s <= t
//     y_t = exp(L_t) S0^T C_t + sum_s P[t][s] x_s + D x_t
//     S_end = exp(L_end) S0 + sum_s e(end, s) dt_s B_s x_s^T
// The four products (scores, C S0, P x, the state's update) run on the matrix cores in float
// (v_mfma_f32_16x16x4_f32: lane l supplies A[l % 16][l / 16] and B[l / 16][l % 16] and holds
// C[4 (l / 16) .. +3][l % 16]).  Four of these instructions in a row take k = 16 i + 4 (l / 16) + j,
// j = 0 .. 3, so that a lane's four operands are 16 consecutive bytes where k runs along a row:
// hence x and S lie transposed in shared memory.  grid: one workgroup per (SC_COLS columns of x,
// head, sequence), in an order that gives each part of the chip consecutive heads (they share B
// and C through that part's cache); eight threads per token of a chunk; the chunk's rows are
// fetched a chunk ahead.
#define SC_COLS 32

typedef __attribute__((__vector_size__(4 * sizeof(float)))) float sc_floatx4_t;

__host__ __device__ inline int sc_padded(int n) { return (n + 15) / 16 * 16; }
__host__ __device__ inline int sc_row_stride(int n) { return sc_padded(n) + 4; }

__device__ __forceinline__ sc_floatx4_t sc_mfma4(float4 a, float4 b, sc_floatx4_t acc) {
    acc = __builtin_amdgcn_mfma_f32_16x16x4f32(a.x, b.x, acc, 0, 0, 0);
    acc = __builtin_amdgcn_mfma_f32_16x16x4f32(a.y, b.y, acc, 0, 0, 0);
    acc = __builtin_amdgcn_mfma_f32_16x16x4f32(a.z, b.z, acc, 0, 0, 0);
    return __builtin_amdgcn_mfma_f32_16x16x4f32(a.w, b.w, acc, 0, 0, 0);
}

// NV: 16-byte loads of B and of C per thread (0: plain loads); NC: the number of states where it
// is known (a multiple of 16: the products' loops are then unrolled), else 0
template <int SC_L, int NV, int NC>
__global__ __launch_bounds__(SC_L * 8) void state_space_chunk_kernel(
        const float* __restrict__ conv, const float* __restrict__ proj,
        const float* __restrict__ A_log, const float* __restrict__ dt_bias,
        const float* __restrict__ skip, float* __restrict__ state, size_t slot_stride,
        const int* __restrict__ q_start, const int* __restrict__ slots, float* __restrict__ out,
        SSShape s, int n_cols, int n_seqs) {
    extern __shared__ __attribute__((aligned(16))) float sc_lds[];
    constexpr int NT = SC_L * 8, NW = NT / 64, TS = SC_L + 4;
    const int N = NC ? NC : s.N;
    const int KS = sc_row_stride(N), Np = sc_padded(N);
    float* Cs = sc_lds;                          // [SC_L][KS]
    float* Bs = Cs + SC_L * KS;                  // [SC_L][KS]
    float* St = Bs + SC_L * KS;                  // [SC_COLS][KS]  S transposed
    float* Xt = St + SC_COLS * KS;               // [SC_COLS][TS]  x transposed
    float* Ps = Xt + SC_COLS * TS;               // [SC_L][TS]
    double* run = (double*)(Ps + SC_L * TS);     // [SC_L]  L_t
    float* dts = (float*)(run + SC_L);           // [SC_L]  dt_t, 0 beyond the chunk's end
    float* wl = dts + SC_L;                      // [SC_L]  e(end, s) dt_s, 0 beyond the chunk's end
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const int li = lane & 15, lg = lane >> 4;
    const int total = n_cols * s.H * n_seqs;
    // workgroups go to the chip's eight parts in turn: part p takes the p-th eighth of the work
    int unit = blockIdx.x;
    if (total % 8 == 0) unit = (unit & 7) * (total >> 3) + (unit >> 3);
    const int col0 = unit % n_cols * SC_COLS;
    const int h = unit / n_cols % s.H, b = unit / (n_cols * s.H);
    const int grp = h / (s.H / s.G), inner = s.H * s.dv;
    const int t0 = q_start[b], t1 = q_start[b + 1];
    if (t0 >= t1) return;                        // the whole workgroup
    float* const S = state + (size_t)slots[b] * slot_stride + (size_t)h * N * s.dv;
    const float rate = expf(A_log[h]), bias = dt_bias[h], Dh = skip[h];
    const int b_col = inner + grp * N, c_col = inner + s.G * N + grp * N, x_col = h * s.dv + col0;

    for (int e = tid; e < Np * SC_COLS; e += NT) {
        const int d = e / SC_COLS, c = e % SC_COLS;
        St[c * KS + d] = (d < N && col0 + c < s.dv) ? S[(size_t)d * s.dv + col0 + c] : 0.f;
    }
    for (int e = tid; e < 2 * SC_L * KS; e += NT) Cs[e] = 0.f;      // B and C: the filling stays zero
    for (int e = tid; e < SC_L * TS; e += NT) Ps[e] = 0.f;          // tiles above the diagonal stay zero

    // eight threads per token fetch its B and C (16 bytes at a time where NV > 0) and its x a chunk
    // ahead, into registers
    const int ft = tid >> 3, sub = tid & 7, n4 = N >> 2;
    float4 rb[NV > 0 ? NV : 1], rc[NV > 0 ? NV : 1];
    float rx[4], rd = 0.f;
    auto fetch = [&](int c0) {
        const int Lc = t1 - c0 < SC_L ? t1 - c0 : SC_L;
        const bool live = ft < Lc;
        const float* cr = conv + (size_t)(c0 + (live ? ft : 0)) * s.conv_width;
#pragma unroll
        for (int i = 0; i < NV; ++i) {
            const int j = sub + 8 * i;
            rb[i] = rc[i] = make_float4(0.f, 0.f, 0.f, 0.f);
            if (live && j < n4) {
                rb[i] = *(const float4*)(cr + b_col + 4 * j);
                rc[i] = *(const float4*)(cr + c_col + 4 * j);
            }
        }
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            const int c = sub * 4 + i;
            rx[i] = (live && col0 + c < s.dv) ? cr[x_col + c] : 0.f;
        }
        if (tid < SC_L)
            rd = tid < Lc ? proj[(size_t)(c0 + tid) * s.row_width + s.dt_off + h] : 0.f;
    };
    fetch(t0);
    for (int c0 = t0; c0 < t1; c0 += SC_L) {
        const int Lc = t1 - c0 < SC_L ? t1 - c0 : SC_L;
        lds_barrier();                           // the chunk before is done with everything
        if (NV > 0) {
#pragma unroll
            for (int i = 0; i < NV; ++i) {
                const int j = sub + 8 * i;
                if (j < n4) {
                    *(float4*)(Bs + ft * KS + 4 * j) = rb[i];
                    *(float4*)(Cs + ft * KS + 4 * j) = rc[i];
                }
            }
        } else {
            const bool live = ft < Lc;
            const float* cr = conv + (size_t)(c0 + (live ? ft : 0)) * s.conv_width;
            for (int e = sub; e < N; e += 8) {
                Bs[ft * KS + e] = live ? cr[b_col + e] : 0.f;
                Cs[ft * KS + e] = live ? cr[c_col + e] : 0.f;
            }
        }
#pragma unroll
        for (int i = 0; i < 4; ++i) Xt[(sub * 4 + i) * TS + ft] = rx[i];
        if (tid < 64) {
            // the first wave: step sizes, and the running sum of the log decays over its lanes
            const bool mine = tid < Lc;
            const float dt = mine ? ss_softplus(rd + bias) : 0.f;
            double sum = -rate * dt;
#pragma unroll
            for (int o = 1; o < SC_L; o <<= 1) {
                const double up = __shfl_up(sum, o, 64);
                if (tid >= o) sum += up;
            }
            const double last = __shfl(sum, SC_L - 1, 64);
            if (tid < SC_L) {
                run[tid] = sum;
                dts[tid] = dt;
                wl[tid] = mine ? expf((float)(last - sum)) * dt : 0.f;
            }
        }
        if (c0 + SC_L < t1) fetch(c0 + SC_L);
        lds_barrier();
        // scores of the chunk, decayed: the 16 x 16 tiles on and below the diagonal, handed out
        // over the waves
        for (int idx = wave; idx < (SC_L / 16) * (SC_L / 16 + 1) / 2; idx += NW) {
            int ti = 0;
            while ((ti + 1) * (ti + 2) / 2 <= idx) ++ti;
            const int si = idx - ti * (ti + 1) / 2;
            sc_floatx4_t acc = {0.f, 0.f, 0.f, 0.f};
            const float* ca = Cs + (ti * 16 + li) * KS + 4 * lg;
            const float* bb = Bs + (si * 16 + li) * KS + 4 * lg;
            const int tr0 = ti * 16 + lg * 4, ss = si * 16 + li;
            const double run_s = run[ss];
            const float dt_s = dts[ss];
            float e[4];
#pragma unroll
            for (int r = 0; r < 4; ++r) e[r] = expf((float)(run[tr0 + r] - run_s)) * dt_s;   // s > t: not used
#pragma unroll 4
            for (int d0 = 0; d0 < Np; d0 += 16)
                acc = sc_mfma4(*(const float4*)(ca + d0), *(const float4*)(bb + d0), acc);
#pragma unroll
            for (int r = 0; r < 4; ++r) Ps[(tr0 + r) * TS + ss] = ss <= tr0 + r ? acc[r] * e[r] : 0.f;
        }
        // the state's share of y for the workgroup's columns: exp(L_t) (C S0)
        sc_floatx4_t num = {0.f, 0.f, 0.f, 0.f};
        const int oti = wave >> 1, oci = wave & 1;
        {
            const float* ca = Cs + (oti * 16 + li) * KS + 4 * lg;
            const float* sb = St + (oci * 16 + li) * KS + 4 * lg;
            float e[4];
#pragma unroll
            for (int r = 0; r < 4; ++r) e[r] = expf((float)run[oti * 16 + lg * 4 + r]);
#pragma unroll 4
            for (int d0 = 0; d0 < Np; d0 += 16)
                num = sc_mfma4(*(const float4*)(ca + d0), *(const float4*)(sb + d0), num);
#pragma unroll
            for (int r = 0; r < 4; ++r) num[r] *= e[r];
        }
        lds_barrier();                           // Ps is whole, St has been read by every wave
        {
            const float* pa = Ps + (oti * 16 + li) * TS + 4 * lg;
            const float* xb = Xt + (oci * 16 + li) * TS + 4 * lg;
            for (int s0 = 0; s0 < (oti + 1) * 16; s0 += 16)
                num = sc_mfma4(*(const float4*)(pa + s0), *(const float4*)(xb + s0), num);
            const int c = oci * 16 + li;
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                const int t = oti * 16 + lg * 4 + r;
                if (t < Lc && col0 + c < s.dv)
                    out[(size_t)(c0 + t) * inner + x_col + c] = fmaf(Dh, Xt[c * TS + t], num[r]);
            }
        }
        // the state after the chunk's last token, transposed: S^T = exp(L_end) S^T + (x w)^T B, a
        // wave's tiles of 16 columns of x by 16 rows of S in turn
        {
            const float aL = expf((float)run[SC_L - 1]);
            for (int tile = wave; tile < (Np / 16) * 2; tile += NW) {
                const int di = tile >> 1, ci = tile & 1;
                sc_floatx4_t acc;
#pragma unroll
                for (int r = 0; r < 4; ++r)
                    acc[r] = aL * St[(ci * 16 + lg * 4 + r) * KS + di * 16 + li];
                const float* xa = Xt + (ci * 16 + li) * TS + 4 * lg;
                const float* bb = Bs + 4 * lg * KS + di * 16 + li;
#pragma unroll
                for (int s0 = 0; s0 < SC_L; s0 += 16) {
                    const float4 xv = *(const float4*)(xa + s0), w = *(const float4*)(wl + s0 + 4 * lg);
                    const float* br = bb + s0 * KS;
                    acc = sc_mfma4(make_float4(xv.x * w.x, xv.y * w.y, xv.z * w.z, xv.w * w.w),
                                   make_float4(br[0], br[KS], br[2 * KS], br[3 * KS]), acc);
                }
#pragma unroll
                for (int r = 0; r < 4; ++r) St[(ci * 16 + lg * 4 + r) * KS + di * 16 + li] = acc[r];
            }
        }
    }
    lds_barrier();
    for (int e = tid; e < N * SC_COLS; e += NT) {
        const int d = e / SC_COLS, c = e % SC_COLS;
        if (col0 + c < s.dv) S[(size_t)d * s.dv + col0 + c] = St[c * KS + d];
    }
}

static int sc_lds_bytes(int N, int L) {
    return (int)sizeof(float) * ((2 * L + SC_COLS) * sc_row_stride(N) + (SC_COLS + L) * (L + 4) + 4 * L);
}

static int sc_lds_limit() {
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

static bool sc_fits(int N, int L) {
    const int bytes = sc_lds_bytes(N, L);
    return bytes <= sc_lds_limit() && bytes <= 160 * 1024;
}

// 1 if the chunked kernel takes these sizes on this device
extern "C" int gfa_state_space_chunks_take(int N, int dv) {
    return N >= 1 && dv >= 1 && sc_fits(N, 32) ? 1 : 0;
}

template <int L, int NV, int NC>
static int sc_launch(const float* conv, const float* proj, const float* A_log, const float* dt_bias,
                     const float* skip, float* state, size_t slot_stride, const int* q_start,
                     const int* slots, float* out, const SSShape& s, int n_seqs, hipStream_t stream) {
    const int bytes = sc_lds_bytes(s.N, L);
    if (bytes > 64 * 1024) {
        static bool allowed = false;
        if (!allowed) {
            const hipError_t e = hipFuncSetAttribute((const void*)state_space_chunk_kernel<L, NV, NC>,
                                                     hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024);
            if (e != hipSuccess) return (int)e;
            allowed = true;
        }
    }
    const int n_cols = (s.dv + SC_COLS - 1) / SC_COLS;
    state_space_chunk_kernel<L, NV, NC><<<n_cols * s.H * n_seqs, L * 8, bytes, stream>>>(
        conv, proj, A_log, dt_bias, skip, state, slot_stride, q_start, slots, out, s, n_cols, n_seqs);
    return GFA_LAUNCH_RESULT();
}

// Chunks of 64 tokens (512 threads) where the device lets a workgroup have the shared memory for
// them and some sequence brings that many, else chunks of 32 (256 threads).
extern "C" int gfa_state_space_chunks(const float* conv, int conv_width, const float* proj, int row_width,
                                      int dt_off, const float* A_log, const float* dt_bias,
                                      const float* skip, float* state, size_t slot_stride,
                                      const int* q_start, const int* slots, float* out, int n_seqs,
                                      int max_q_len, int H, int G, int N, int dv, hipStream_t stream) {
    if (n_seqs <= 0) return 0;
    SSShape s{H, G, N, dv, conv_width, row_width, dt_off};
    if (!ss_fits(s, n_seqs) || !gfa_state_space_chunks_take(N, dv) ||
            (long long)((dv + SC_COLS - 1) / SC_COLS) * H * n_seqs > 0x7fffffffLL)
        return (int)hipErrorInvalidValue;
    // 16-byte loads of B and C where every row and group starts at a multiple of four floats
    const bool vec = N % 4 == 0 && conv_width % 4 == 0 && (H * dv) % 4 == 0 && (size_t)conv % 16 == 0
        && N <= 256;
    const bool big = max_q_len > 32 && sc_fits(N, 64);
#define SC_GO(NV, NC) return big ? sc_launch<64, NV, NC>(conv, proj, A_log, dt_bias, skip, state, slot_stride, \
                                                       q_start, slots, out, s, n_seqs, stream) \
                                 : sc_launch<32, NV, NC>(conv, proj, A_log, dt_bias, skip, state, slot_stride, \
                                                       q_start, slots, out, s, n_seqs, stream)
    if (!vec) SC_GO(0, 0);
    if (N == 64) SC_GO(2, 64);
    if (N == 128) SC_GO(4, 128);
    if (N <= 64) SC_GO(2, 0);
    if (N <= 128) SC_GO(4, 0);
    SC_GO(8, 0);
#undef SC_GO
}
