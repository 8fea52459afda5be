// mlstm.hip — the matrix-memory recurrence (mLSTM of the xLSTM family), token by token with the state in registers.
//
// Per head: a state matrix S [dim][vdim], a normaliser n [dim] and a running maximum m of the log gates, all f32, one set per sequence slot.  For a token
// with query q (already scaled by dim^-1/2 here), key k, value v and the pre-activations of the two gates:
//     i = cap tanh(i_pre / cap)            f = logsigmoid(cap tanh(f_pre / cap))        (both made for the whole batch at once: launch_mlstm_gates)
//     m' = max(f + m, i)     S' = e^(f + m - m') S + e^(i - m') k v^T     n' likewise with k alone
//     o  = S'^T q / (max(|n' . q|, e^(-m')) + 1e-6)
// A state that has seen nothing is S = 0, n = 0, m = 0.  The columns of S evolve independently given the gates, so a workgroup owns 64 columns of one head of
// one sequence segment: lane = column, the 8 or 16 waves split the dim rows (each thread keeps its rows of its column - and of n - in registers), the per-token
// partial sums of S^T q and n . q cross the waves through LDS.  A segment is a run of consecutive rows of the batch that belong to one sequence: a prompt,
// a portion of one, or a single decoded token - the same code, started from the slot's state and ending with the state written back.
//
// Three forms of the same recurrence, by what a launch's segments hold.  A token's weight in what a later token reads depends on the gates alone: with
// F_t = f_1 + .. + f_t inside a chunk of 64 tokens and m_0, S_0 in front of it
//     S_t = e^(F_t + m_0 - m_t) S_0 + sum_(s <= t) e^(F_t - F_s + i_s - m_t) k_s v_s^T        m_t = F_t + max(m_0, max_(s <= t) (i_s - F_s))
// * mlstm_step  - every segment is one row (a decode step): gates, update and read-out in one launch, each entry of S touched once on its way through.
// * mlstm_chunk - long segments: mlstm_log_gates makes i, F (double) and m of all tokens (prefix sums and maxima over lanes), mlstm_scores the weighted products
//                 q_t . k_s of every chunk at once, and mlstm_chunk walks the chunks with S in registers: o = e^.. S_0^T q + W V, S <- e^.. S_0 + K^T (u V).  All
//                 products on the f32 matrix cores (v_mfma_f32_16x16x4_f32).  n is one more column whose values are 1; the division is left to mlstm_out.
// * mlstm_scan  - everything else, token by token as described above.
// The state of a slot holds a copy of n and of m per 64-column block: the column blocks of one head run as workgroups of their own, and each reads and writes
// its copy only (mlstm_state_copies).
//
// mlstm_out: per head, the output divided by its root mean square, times the mixer's norm weight (per head and entry, one vector shared by the heads, or none), times
// sigmoid - or silu - of the output gate's pre-activation.  The delta-rule mixers close with the same launch.
#include "kernels.h"

namespace mi355 {

namespace {

typedef float f32x4 __attribute__((ext_vector_type(4)));

template <int DPER, int NDG>
__global__ __launch_bounds__(64 * NDG) void mlstm_scan_kernel(MlstmArgs a) {
    // CH tokens' inputs are staged in LDS by the whole workgroup at once - one trip to memory per CH tokens instead of one per token in the dependency
    // chain - and the recurrence then runs out of LDS and registers
    constexpr int DP = NDG * DPER, CH = 2048 / DP, NT = 64 * NDG;
    __shared__ float sq[CH][DP], sk[CH][DP], sv[CH][64], sg[CH][2], red[2][NDG][64], redn[2][NDG];
    const int seg = blockIdx.x, h = blockIdx.y, tid = threadIdx.x, j = tid & 63, dg = tid >> 6;
    const int col = blockIdx.z * 64 + j, d0 = dg * DPER;
    const int H = a.H, D = a.D, VD = a.VD;
    const int start = a.seg_start[seg], len = a.seg_len[seg], slot = a.seg_slot[seg];
    float *Sg = a.S + ((size_t)slot * H + h) * (size_t)D * VD;
    const int NZ = gridDim.z;
    float *ng = a.n + (((size_t)slot * H + h) * NZ + blockIdx.z) * D;
    float *mg = a.m + ((size_t)slot * H + h) * NZ + blockIdx.z;
    float S[DPER], n[DPER];
#pragma unroll
    for (int e = 0; e < DPER; e++) {
        const int d = d0 + e;
        S[e] = d < D && col < VD ? Sg[(size_t)d * VD + col] : 0.0f;
        n[e] = d < D ? ng[d] : 0.0f;
    }
    float m = *mg;
    const float qscale = 1.0f / sqrtf((float)D);
    const int off_k = H * D, off_v = 2 * H * D, off_i = 2 * H * D + 2 * H * VD, off_f = off_i + H;
    for (int t0 = 0; t0 < len; t0 += CH) {
        const int nc = len - t0 < CH ? len - t0 : CH;
        __syncthreads();                                        // (the previous chunk has been used up)
        for (int idx = tid; idx < nc * DP; idx += NT) {
            const int tt = idx / DP, d = idx - tt * DP;
            const float *row = a.p + (size_t)(start + t0 + tt) * a.ld_p;
            sq[tt][d] = d < D ? row[h * D + d] * qscale : 0.0f;
            sk[tt][d] = d < D ? row[off_k + h * D + d] : 0.0f;
        }
        for (int idx = tid; idx < nc * 64; idx += NT) {
            const int tt = idx >> 6, c = blockIdx.z * 64 + (idx & 63);
            sv[tt][idx & 63] = c < VD ? a.p[(size_t)(start + t0 + tt) * a.ld_p + off_v + h * VD + c] : 0.0f;
        }
        if (tid < nc * 2) sg[tid >> 1][tid & 1] = a.p[(size_t)(start + t0 + (tid >> 1)) * a.ld_p + ((tid & 1) ? off_f : off_i) + h];   // log gates (mlstm_gates_kernel)
        __syncthreads();
        for (int tt = 0; tt < nc; tt++) {
            const float v = sv[tt][j], ig = sg[tt][0], fg = sg[tt][1];
            const float mn = fmaxf(fg + m, ig), ea = expf(fg + m - mn), eb = expf(ig - mn);
            m = mn;
            float num = 0.0f, nq = 0.0f;
#pragma unroll
            for (int e = 0; e < DPER; e++) {
                const float kd = eb * sk[tt][d0 + e], q = sq[tt][d0 + e];
                S[e] = fmaf(ea, S[e], kd * v);
                n[e] = fmaf(ea, n[e], kd);
                num = fmaf(S[e], q, num);
                nq = fmaf(n[e], q, nq);
            }
            const int pb = tt & 1;                              // (two sets of partial sums: one barrier per token is enough)
            red[pb][dg][j] = num;
            if (j == 0) redn[pb][dg] = nq;
            __syncthreads();
            if (dg == 0 && col < VD) {
                float nt = 0.0f, qt = 0.0f;
#pragma unroll
                for (int w = 0; w < NDG; w++) { nt += red[pb][w][j]; qt += redn[pb][w]; }
                a.o[(size_t)(start + t0 + tt) * a.ld_o + (size_t)h * VD + col] = nt / (fmaxf(fabsf(qt), expf(-m)) + 1e-6f);
            }
        }
    }
#pragma unroll
    for (int e = 0; e < DPER; e++) {
        const int d = d0 + e;
        if (d < D && col < VD) Sg[(size_t)d * VD + col] = S[e];
        if (d < D && j == 0) ng[d] = n[e];
    }
    if (tid == 0) *mg = m;
}

__device__ __forceinline__ float mlstm_log_sigmoid(float z) { return fminf(z, 0.0f) - log1pf(expf(-fabsf(z))); }
__device__ __forceinline__ float mlstm_cap(float z, float cap) { return cap * tanhf(z / cap); }

// ---------------------------------------------------------------- single rows
// a workgroup owns 64 columns of one head of one segment: lane = column, the waves share the rows; wave 0 also brings n and its product with q
constexpr int MLS_NW = 8;
__global__ __launch_bounds__(64 * MLS_NW) void mlstm_step_kernel(MlstmArgs a) {
    __shared__ float red[MLS_NW][64];
    const int seg = blockIdx.x, h = blockIdx.y, lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
    const int col = blockIdx.z * 64 + lane, NZ = gridDim.z;
    const int H = a.H, D = a.D, VD = a.VD, row = a.row0 + seg, slot = a.seg_slot[seg];   // (single rows side by side)
    const float *p = a.p + (size_t)row * a.ld_p, *q = p + h * D, *k = p + (H + h) * D;
    float *Sg = a.S + ((size_t)slot * H + h) * (size_t)D * VD + col;
    float *ng = a.n + (((size_t)slot * H + h) * NZ + blockIdx.z) * D, *mg = a.m + ((size_t)slot * H + h) * NZ + blockIdx.z;
    const int off_v = 2 * H * D, off_i = off_v + 2 * H * VD;
    const bool in = col < VD;
    const float v = in ? p[off_v + h * VD + col] : 0.0f, m0 = *mg;
    const float ig = mlstm_cap(p[off_i + h] + (a.i_bias ? a.i_bias[h] : 0.0f), a.gate_cap);
    const float fg = mlstm_log_sigmoid(mlstm_cap(p[off_i + H + h] + (a.f_bias ? a.f_bias[h] : 0.0f), a.gate_cap));
    const float m = fmaxf(fg + m0, ig), ea = expf(fg + m0 - m), eb = expf(ig - m), qscale = 1.0f / sqrtf((float)D);
    float num = 0.0f, nq = 0.0f;
#pragma unroll 16
    for (int d = wave; d < D; d += MLS_NW) {
        const float s = fmaf(ea, in ? Sg[(size_t)d * VD] : 0.0f, eb * k[d] * v);
        if (in) Sg[(size_t)d * VD] = s;
        num = fmaf(s, q[d] * qscale, num);
    }
    red[wave][lane] = num;
    if (wave == 0) {
        for (int d = lane; d < D; d += 64) {
            const float n = fmaf(ea, ng[d], eb * k[d]);
            ng[d] = n;
            nq = fmaf(n, q[d] * qscale, nq);
        }
#pragma unroll
        for (int o = 32; o > 0; o >>= 1) nq += __shfl_xor(nq, o, 64);
    }
    __syncthreads();
    if (wave != 0) return;
    float t = 0.0f;
#pragma unroll
    for (int w = 0; w < MLS_NW; w++) t += red[w][lane];
    if (in) a.o[(size_t)row * a.ld_o + (size_t)h * VD + col] = t / (fmaxf(fabsf(nq), expf(-m)) + 1e-6f);
    if (lane == 0) *mg = m;
}

// ---------------------------------------------------------------- long segments, chunks of 64 tokens
constexpr int MLC_T = 64;

// i (in place), F, m of every token and m in front of every chunk (at the chunk's first row); the slot's m moves on.  A wave per chunk, 8 chunks at a time
__global__ __launch_bounds__(512) void mlstm_log_gates_kernel(MlstmArgs a, int NZ) {
    __shared__ double tot[8];
    __shared__ double top[8];
    const int seg = blockIdx.x, h = blockIdx.y, lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    const int H = a.H, start = a.seg_start[seg], len = a.seg_len[seg], slot = a.seg_slot[seg], off_i = 2 * H * a.D + 2 * H * a.VD;
    float *mg = a.m + ((size_t)slot * H + h) * NZ;
    float m_in = *mg;
    const float ib = a.i_bias ? a.i_bias[h] : 0.0f, fb = a.f_bias ? a.f_bias[h] : 0.0f;
    for (int t0 = 0; t0 < len; t0 += 8 * MLC_T) {
        const int t = t0 + wave * MLC_T + lane, row = start + t;
        const bool live = t < len;
        float *g = const_cast<float *>(a.p) + (size_t)(live ? row : start) * a.ld_p + off_i;
        const float ig = live ? mlstm_cap(g[h] + ib, a.gate_cap) : 0.0f;
        double F = live ? (double)mlstm_log_sigmoid(mlstm_cap(g[H + h] + fb, a.gate_cap)) : 0.0;
#pragma unroll
        for (int o = 1; o < 64; o <<= 1) { const double u = __shfl_up(F, o, 64); if (lane >= o) F += u; }
        double x = live ? (double)ig - F : -1e300;
#pragma unroll
        for (int o = 1; o < 64; o <<= 1) { const double u = __shfl_up(x, o, 64); if (lane >= o) x = u > x ? u : x; }
        if (lane == 63) { tot[wave] = F; top[wave] = x; }       // (rows past the end add nothing to either)
        __syncthreads();
        float m0 = m_in;
        for (int w = 0; w < 8; w++) {
            if (w == wave) m0 = m_in;
            const double y = (double)m_in > top[w] ? (double)m_in : top[w];
            m_in = (float)(tot[w] + y);
        }
        if (live) {
            const double y = (double)m0 > x ? (double)m0 : x;
            const size_t at = (size_t)row * H + h;
            g[h] = ig;
            a.w_F[at] = F; a.w_m[at] = (float)(F + y);
            if (lane == 0) a.w_m0[at] = m0;
        }
        __syncthreads();                                        // (tot and top have been read)
    }
    if (threadIdx.x < NZ) mg[threadIdx.x] = m_in;
}

// W[row t][h][s] = e^(F_t - F_s + i_s - m_t) (q_t . k_s) / sqrt(dim), s <= t inside t's chunk, 0 where the chunk's rows end; tiles above the diagonal stay unwritten
__global__ __launch_bounds__(256) void mlstm_scores_kernel(MlstmArgs a, int chunks) {
    __shared__ double F[MLC_T];
    __shared__ float ig[MLC_T], mt[MLC_T];
    const int seg = blockIdx.x / chunks, c = blockIdx.x - seg * chunks, h = blockIdx.y, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, l16 = lane & 15, lg = lane >> 4;
    const int H = a.H, D = a.D, len = a.seg_len[seg] - c * MLC_T, row0 = a.seg_start[seg] + c * MLC_T;
    if (len <= 0) return;                                       // (uniform: before the barrier)
    const int nc = len < MLC_T ? len : MLC_T, off_i = 2 * H * D + 2 * H * a.VD;
    if (tid < MLC_T) {
        const int r = row0 + (tid < nc ? tid : 0);
        F[tid] = a.w_F[(size_t)r * H + h]; mt[tid] = a.w_m[(size_t)r * H + h]; ig[tid] = a.p[(size_t)r * a.ld_p + off_i + h];
    }
    const int t = 16 * wave + l16;
    const float *q = a.p + (size_t)(row0 + (t < nc ? t : nc - 1)) * a.ld_p + h * D;
    const float *k[4];
    f32x4 acc[4];
#pragma unroll
    for (int u = 0; u < 4; u++) {
        const int s = 16 * u + l16;
        k[u] = a.p + (size_t)(row0 + (s < nc ? s : nc - 1)) * a.ld_p + (H + h) * D;
        acc[u] = f32x4{0.0f, 0.0f, 0.0f, 0.0f};
    }
#pragma unroll 2
    for (int d0 = 0; d0 < D; d0 += 16) {
        const int d = d0 + 4 * lg;
        const bool in = d < D;
        const f32x4 zero = {0.0f, 0.0f, 0.0f, 0.0f}, q4 = in ? *reinterpret_cast<const f32x4 *>(q + d) : zero;
        f32x4 k4[4];
#pragma unroll
        for (int u = 0; u < 4; u++) k4[u] = in ? *reinterpret_cast<const f32x4 *>(k[u] + d) : zero;
#pragma unroll
        for (int u = 0; u < 4; u++) {
            if (u > wave) continue;
#pragma unroll
            for (int e = 0; e < 4; e++) acc[u] = __builtin_amdgcn_mfma_f32_16x16x4f32(k4[u][e], q4[e], acc[u], 0, 0, 0);
        }
    }
    __syncthreads();
    if (t >= nc) return;
    const float qscale = 1.0f / sqrtf((float)D);
    float *W = a.w_A + ((size_t)(row0 + t) * H + h) * MLC_T;
#pragma unroll
    for (int u = 0; u < 4; u++) {
        if (u > wave) continue;
        f32x4 o;
#pragma unroll
        for (int r = 0; r < 4; r++) {
            const int s = 16 * u + 4 * lg + r;
            o[r] = s <= t ? expf((float)(F[t] - F[s] + (double)ig[s] - (double)mt[t])) * (acc[u][r] * qscale) : 0.0f;   // (s <= t < nc)
        }
        *reinterpret_cast<f32x4 *>(W + 16 * u + 4 * lg) = o;
    }
}

// 16 columns of one head of one segment (the last block: the column of ones, n).  Four waves; wave w finishes tokens 16 w .. + 15 of every chunk and keeps rows
// 16 DTW w .. + 16 DTW - 1 of S.  S in the matrix cores' result layout: lane = (column l & 15), register r of tile i = row 16 (DTW w + i) + 4 (l >> 4) + r; a
// copy by columns in LDS is what the read-out multiplies.  The next chunk's q, k, v and W rows are on their way while a chunk is worked on.
template <int DTW>
__global__ __launch_bounds__(256) void mlstm_chunk_kernel(MlstmArgs a, int NZ) {
    constexpr int DT = 4 * DTW, LDT = 16 * DT + 4, LDV = MLC_T + 4;
    __shared__ __attribute__((aligned(16))) float St[16][LDT], Vt[16][LDV];
    __shared__ __attribute__((aligned(16))) float wu[MLC_T], wi[MLC_T];
    const int seg = blockIdx.x, h = blockIdx.y, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, l16 = lane & 15, lg = lane >> 4;
    const int H = a.H, D = a.D, VD = a.VD, NCB = (VD + 15) >> 4;
    const bool ones = (int)blockIdx.z == NCB;
    const int col = blockIdx.z * 16 + l16;
    const bool cin = ones ? l16 == 0 : col < VD;
    const int start = a.seg_start[seg], len = a.seg_len[seg], slot = a.seg_slot[seg];
    const int off_k = (H + h) * D, off_v = 2 * H * D + h * VD, off_i = 2 * H * D + 2 * H * VD + h;
    float *Sg = ones ? a.n + ((size_t)slot * H + h) * NZ * D : a.S + ((size_t)slot * H + h) * (size_t)D * VD + col;
    const size_t sstride = ones ? 1 : VD;
    const float qscale = 1.0f / sqrtf((float)D);
    f32x4 S[DTW];
#pragma unroll
    for (int i = 0; i < DTW; i++) {
#pragma unroll
        for (int r = 0; r < 4; r++) {
            const int d = 16 * (DTW * wave + i) + 4 * lg + r;
            S[i][r] = cin && d < D ? Sg[(size_t)d * sstride] : 0.0f;
        }
        *reinterpret_cast<f32x4 *>(&St[l16][16 * (DTW * wave + i) + 4 * lg]) = S[i];
    }
    f32x4 nq[DT], nA[4], nv;
    float nk[DTW][16], ni = 0.0f, nm = 0.0f;
    double nFd = 0.0, nFT = 0.0;
    float nmT = 0.0f, nm0 = 0.0f;
    const auto request = [&](int t0) {
        const int nc = len - t0 < MLC_T ? len - t0 : MLC_T, row0 = start + t0;
        const int t = 16 * wave + l16;
        const size_t tr = (size_t)(row0 + (t < nc ? t : nc - 1));
        const float *q = a.p + tr * a.ld_p + h * D, *A = a.w_A + (tr * H + h) * MLC_T;
#pragma unroll
        for (int u = 0; u < DT; u++) nq[u] = 16 * u + 4 * lg < D ? *reinterpret_cast<const f32x4 *>(q + 16 * u + 4 * lg) : f32x4{0.0f, 0.0f, 0.0f, 0.0f};
#pragma unroll
        for (int u = 0; u < 4; u++) nA[u] = u <= wave ? *reinterpret_cast<const f32x4 *>(A + 16 * u + 4 * lg) : f32x4{0.0f, 0.0f, 0.0f, 0.0f};
#pragma unroll
        for (int j = 0; j < 16; j++) {
            const int s = 16 * (j >> 2) + 4 * lg + (j & 3);
            const float *k = a.p + (size_t)(row0 + (s < nc ? s : nc - 1)) * a.ld_p + off_k;
#pragma unroll
            for (int i = 0; i < DTW; i++) { const int d = 16 * (DTW * wave + i) + l16; nk[i][j] = d < D ? k[d] : 0.0f; }
        }
        const int s = tid >> 2, c4 = (tid & 3) * 4;
#pragma unroll
        for (int e = 0; e < 4; e++) {
            const int c = blockIdx.z * 16 + c4 + e;
            nv[e] = s >= nc ? 0.0f : ones ? (c4 + e == 0 ? 1.0f : 0.0f) : c < VD ? a.p[(size_t)(row0 + s) * a.ld_p + off_v + c] : 0.0f;
        }
        const size_t last = (size_t)(row0 + nc - 1) * H + h;
        nFT = a.w_F[last]; nmT = a.w_m[last]; nm0 = a.w_m0[(size_t)row0 * H + h];
        if (tid < MLC_T) {
            const size_t at = (size_t)(row0 + (tid < nc ? tid : nc - 1)) * H + h;
            nFd = a.w_F[at]; nm = a.w_m[at]; ni = a.p[(size_t)(row0 + (tid < nc ? tid : nc - 1)) * a.ld_p + off_i];
        }
    };
    request(0);
    for (int t0 = 0; t0 < len; t0 += MLC_T) {
        const int nc = len - t0 < MLC_T ? len - t0 : MLC_T, row0 = start + t0;
        f32x4 q[DT], A[4];
        float k[DTW][16];
#pragma unroll
        for (int u = 0; u < DT; u++) q[u] = nq[u];
#pragma unroll
        for (int u = 0; u < 4; u++) A[u] = nA[u];
#pragma unroll
        for (int i = 0; i < DTW; i++)
#pragma unroll
            for (int j = 0; j < 16; j++) k[i][j] = nk[i][j];
#pragma unroll
        for (int e = 0; e < 4; e++) Vt[(tid & 3) * 4 + e][tid >> 2] = nv[e];
        const float g = expf((float)(nFT + (double)nm0 - (double)nmT));
        if (tid < MLC_T) {
            wu[tid] = expf((float)(nFT - nFd + (double)ni - (double)nmT));          // (rows past the end: values 0)
            wi[tid] = expf((float)(nFd + (double)nm0 - (double)nm)) * qscale;
        }
        __syncthreads();
        if (t0 + MLC_T < len) request(t0 + MLC_T);
        // ---- outputs of this wave's 16 tokens
        f32x4 acc = {0.0f, 0.0f, 0.0f, 0.0f};
#pragma unroll
        for (int u = 0; u < DT; u++) {
            const f32x4 s4 = *reinterpret_cast<const f32x4 *>(&St[l16][16 * u + 4 * lg]);
#pragma unroll
            for (int e = 0; e < 4; e++) acc = __builtin_amdgcn_mfma_f32_16x16x4f32(q[u][e], s4[e], acc, 0, 0, 0);
        }
        const f32x4 w4 = *reinterpret_cast<const f32x4 *>(&wi[16 * wave + 4 * lg]);
        acc.x *= w4.x; acc.y *= w4.y; acc.z *= w4.z; acc.w *= w4.w;
        f32x4 v4[4];
#pragma unroll
        for (int u = 0; u < 4; u++) v4[u] = *reinterpret_cast<const f32x4 *>(&Vt[l16][16 * u + 4 * lg]);
#pragma unroll
        for (int u = 0; u < 4; u++) {
            if (u > wave) continue;
#pragma unroll
            for (int e = 0; e < 4; e++) acc = __builtin_amdgcn_mfma_f32_16x16x4f32(A[u][e], v4[u][e], acc, 0, 0, 0);
        }
#pragma unroll
        for (int r = 0; r < 4; r++) {
            const int t = 16 * wave + 4 * lg + r;
            if (t < nc && cin) {
                if (ones) a.w_nq[(size_t)(row0 + t) * H + h] = acc[r];
                else a.o[(size_t)(row0 + t) * a.ld_o + (size_t)h * VD + col] = acc[r];
            }
        }
        // ---- the state behind the chunk
#pragma unroll
        for (int u = 0; u < 4; u++) {
            const f32x4 u4 = *reinterpret_cast<const f32x4 *>(&wu[16 * u + 4 * lg]);
            v4[u].x *= u4.x; v4[u].y *= u4.y; v4[u].z *= u4.z; v4[u].w *= u4.w;
        }
#pragma unroll
        for (int i = 0; i < DTW; i++) {
            S[i].x *= g; S[i].y *= g; S[i].z *= g; S[i].w *= g;
#pragma unroll
            for (int j = 0; j < 16; j++) S[i] = __builtin_amdgcn_mfma_f32_16x16x4f32(k[i][j], v4[j >> 2][j & 3], S[i], 0, 0, 0);
        }
        __syncthreads();                                        // (everyone has read the old state and this chunk's values)
#pragma unroll
        for (int i = 0; i < DTW; i++) *reinterpret_cast<f32x4 *>(&St[l16][16 * (DTW * wave + i) + 4 * lg]) = S[i];
    }
#pragma unroll
    for (int i = 0; i < DTW; i++)
#pragma unroll
        for (int r = 0; r < 4; r++) {
            const int d = 16 * (DTW * wave + i) + 4 * lg + r;
            if (!cin || d >= D) continue;
            if (ones) for (int z = 0; z < NZ; z++) Sg[(size_t)z * D + d] = S[i][r];
            else Sg[(size_t)d * sstride] = S[i][r];
        }
}

// the two log gates of every (token, head), in place over their pre-activations: i = cap tanh((x + b_i) / cap), f = logsigmoid(cap tanh((x + b_f) / cap))
__global__ void mlstm_gates_kernel(float *p, int ld_p, int off_i, int H, int T, const float *ib, const float *fb, float cap) {
    const int i = blockIdx.x * blockDim.x + threadIdx.x;
    if (i >= T * H) return;
    const int t = i / H, h = i - t * H;
    float *row = p + (size_t)t * ld_p + off_i;
    const float ig = cap * tanhf((row[h] + (ib ? ib[h] : 0.0f)) / cap);
    const float fz = cap * tanhf((row[H + h] + (fb ? fb[h] : 0.0f)) / cap);
    row[h] = ig;
    row[H + h] = fminf(fz, 0.0f) - log1pf(expf(-fabsf(fz)));
}

__global__ __launch_bounds__(64) void mlstm_out_kernel(const float *o, int ld_o, const float *p, int ld_p, int off_g, const float *w, int H, int VD, float eps,
                                                       float *y, int ld_y, int w_stride, int gate, const float *nq, const float *m) {
    const int t = blockIdx.x, h = blockIdx.y, lane = threadIdx.x;
    const float *orow = o + (size_t)t * ld_o + (size_t)h * VD;
    float ss = 0.0f;
    for (int i = lane; i < VD; i += 64) { const float v = orow[i]; ss = fmaf(v, v, ss); }
#pragma unroll
    for (int s = 32; s > 0; s >>= 1) ss += __shfl_xor(ss, s, 64);
    // (nq: the outputs still lack their denominator max(|n . q|, e^-m) + 1e-6)
    const float den = nq ? 1.0f / (fmaxf(fabsf(nq[(size_t)t * H + h]), expf(-m[(size_t)t * H + h])) + 1e-6f) : 1.0f;
    const float inv = nq ? den / sqrtf((ss * den) * den / (float)VD + eps) : 1.0f / sqrtf(ss / (float)VD + eps);
    for (int i = lane; i < VD; i += 64) {
        const float g = p[(size_t)t * ld_p + off_g + h * VD + i];
        const float sg = 1.0f / (1.0f + expf(-g));
        y[(size_t)t * ld_y + (size_t)h * VD + i] = orow[i] * inv * (w ? w[h * w_stride + i] : 1.0f) * (gate == MLSTM_GATE_SILU ? g * sg : sg);
    }
}

__global__ void mlstm_state_reset_kernel(float *S, size_t n_s, float *n, size_t n_n, float *m, size_t n_m) {
    const size_t i = (size_t)blockIdx.x * blockDim.x + threadIdx.x;
    if (i < n_s) S[i] = 0.0f;
    if (i < n_n) n[i] = 0.0f;
    if (i < n_m) m[i] = 0.0f;
}

}  // namespace

bool mlstm_shape_ok(int D, int VD) { return D >= 1 && D <= 512 && VD >= 1; }
int mlstm_state_copies(int VD) { return (VD + 63) / 64; }

hipError_t launch_mlstm(const MlstmArgs &a, int T, bool *divided, hipStream_t st) {
    *divided = true;
    if (a.n_seg <= 0 || T <= 0) return hipSuccess;
    if (!mlstm_shape_ok(a.D, a.VD) || !(a.gate_cap > 0.0f)) return hipErrorInvalidValue;
    const int NZ = mlstm_state_copies(a.VD);
    const dim3 grid((unsigned)a.n_seg, (unsigned)a.H, (unsigned)NZ);
    if (a.max_len == 1) {
        hipLaunchKernelGGL(mlstm_step_kernel, grid, dim3(64 * MLS_NW), 0, st, a);
        return hipGetLastError();
    }
    const bool vec = (a.D & 3) == 0 && (a.ld_p & 3) == 0 && (reinterpret_cast<uintptr_t>(a.p) & 15) == 0;
    if (a.max_len >= MLSTM_CHUNK_MIN_ROWS && vec && NZ <= 512 && a.w_A && a.w_F && a.w_m && a.w_m0 && a.w_nq) {
        *divided = false;
        const int chunks = (a.max_len + MLC_T - 1) / MLC_T;
        hipLaunchKernelGGL(mlstm_log_gates_kernel, dim3((unsigned)a.n_seg, (unsigned)a.H), dim3(512), 0, st, a, NZ);
        hipLaunchKernelGGL(mlstm_scores_kernel, dim3((unsigned)(a.n_seg * chunks), (unsigned)a.H), dim3(256), 0, st, a, chunks);
        const dim3 cg((unsigned)a.n_seg, (unsigned)a.H, (unsigned)((a.VD + 15) / 16 + 1));
        if (a.D <= 64) hipLaunchKernelGGL(mlstm_chunk_kernel<1>, cg, dim3(256), 0, st, a, NZ);
        else if (a.D <= 128) hipLaunchKernelGGL(mlstm_chunk_kernel<2>, cg, dim3(256), 0, st, a, NZ);
        else if (a.D <= 256) hipLaunchKernelGGL(mlstm_chunk_kernel<4>, cg, dim3(256), 0, st, a, NZ);
        else hipLaunchKernelGGL(mlstm_chunk_kernel<8>, cg, dim3(256), 0, st, a, NZ);
        return hipGetLastError();
    }
    hipLaunchKernelGGL(mlstm_gates_kernel, dim3((unsigned)((T * a.H + 255) / 256)), dim3(256), 0, st, const_cast<float *>(a.p) + (size_t)a.row0 * a.ld_p, a.ld_p,
                       2 * a.H * a.D + 2 * a.H * a.VD, a.H, T, a.i_bias, a.f_bias, a.gate_cap);
    // dim rows per thread x waves per workgroup: the waves of a workgroup split the rows of the state, the more of them the shorter a token's chain
    if (a.D <= 16) hipLaunchKernelGGL((mlstm_scan_kernel<2, 8>), grid, dim3(512), 0, st, a);
    else if (a.D <= 32) hipLaunchKernelGGL((mlstm_scan_kernel<4, 8>), grid, dim3(512), 0, st, a);
    else if (a.D <= 64) hipLaunchKernelGGL((mlstm_scan_kernel<8, 8>), grid, dim3(512), 0, st, a);
    else if (a.D <= 128) hipLaunchKernelGGL((mlstm_scan_kernel<8, 16>), grid, dim3(1024), 0, st, a);
    else if (a.D <= 256) hipLaunchKernelGGL((mlstm_scan_kernel<16, 16>), grid, dim3(1024), 0, st, a);
    else hipLaunchKernelGGL((mlstm_scan_kernel<32, 16>), grid, dim3(1024), 0, st, a);
    return hipGetLastError();
}

hipError_t launch_mlstm_out(const float *o, int ld_o, const float *p, int ld_p, int off_g, const float *w, int T, int H, int VD, float eps, float *y, int ld_y,
                            hipStream_t st, int w_stride, int gate, const float *nq, const float *m) {
    if (T <= 0) return hipSuccess;
    if (nq && !m) return hipErrorInvalidValue;
    hipLaunchKernelGGL(mlstm_out_kernel, dim3((unsigned)T, (unsigned)H), dim3(64), 0, st, o, ld_o, p, ld_p, off_g, w, H, VD, eps, y, ld_y, w_stride < 0 ? VD : w_stride, gate, nq, m);
    return hipGetLastError();
}

hipError_t launch_mlstm_state_reset(float *S, size_t n_s, float *n, size_t n_n, float *m, size_t n_m, hipStream_t st) {
    const size_t mx = n_s > n_n ? (n_s > n_m ? n_s : n_m) : (n_n > n_m ? n_n : n_m);
    if (!mx) return hipSuccess;
    hipLaunchKernelGGL(mlstm_state_reset_kernel, dim3((unsigned)((mx + 255) / 256)), dim3(256), 0, st, S, n_s, n, n_n, m, n_m);
    return hipGetLastError();
}

}  // namespace mi355
