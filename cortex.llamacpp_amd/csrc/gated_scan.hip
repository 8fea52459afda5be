// gated_scan.hip — linear recurrences with a learned decay and no softmax: per head a state S [D][VD], f32, one per sequence slot; for a token with query q, key k,
// value v
//     S <- diag(a) S + k v^T            o = S^T q  (+ skip v)
// The decay a is one number per key channel (gated linear attention; a = sigmoid(z)^(1/tau), z from a low-rank projection) or one per head (Mamba-2's state-space
// form; a = exp(-exp(A_log) dt), dt = softplus(pre + bias), and the key counts dt times).  Heads may share queries and keys in groups of neighbours.
//
// Two forms of the same recurrence, by what a launch's segments hold (a segment: a run of consecutive batch rows of one sequence; it starts from the slot's
// state and leaves the state behind, so the result does not depend on how a sequence was cut):
// * gated_step - every segment is one row (a decode step): decays, the optional short convolution in front of q / k / v, update, read-out - and for states of up to
//   256 columns the per-head unit norm and the output gate - in one launch; each entry of S is touched once on its way through.
// * chunks of 64 tokens - everything else.  A token's weight in what a later token reads is a product of decays; inside a chunk
//       o_t = (q_t P_t)^T S_0 + sum_(s <= t) A_ts v_s      P_t = a_1 .. a_t      A_ts = sum_d q_td k_sd (a_(s+1) .. a_t)_d
//       S   = diag(P_end) S_0 + sum_s (k_s a_(s+1) .. a_end) v_s^T
//   All factors are PRODUCTS of decays over the tokens between - never a quotient of two prefix products and never an exponent's difference, so a decay that
//   closes (a = 0) or a long chunk of small ones underflows to the zero it stands for.  Everything but the walk from
//   chunk to chunk is made for all chunks at once: A with the scaled q and k (gated_intra_*), what a chunk adds to the state (gated_update), and the outputs
//   (gated_out); the walk itself touches every entry of the state once per chunk (gated_carry) and leaves the state in front of the chunk in the place of what the
//   chunk adds.  The products of update and outputs, and A of the one-decay form, run on the f32 matrix cores (v_mfma_f32_16x16x4_f32).
//
// conv_silu: the short causal convolution over time with bias and silu in front of a batch (steps do it inside).  gated_norm: y = o silu(z) over its root mean
// square in equal parts, times a weight.
#include "kernels.h"

namespace mi355 {

namespace {

typedef float f32x4 __attribute__((ext_vector_type(4)));

__device__ __forceinline__ float gs_softplus(float z) { return fmaxf(z, 0.0f) + log1pf(expf(-fabsf(z))); }
__device__ __forceinline__ float gs_silu(float z) { return z / (1.0f + expf(-z)); }
__device__ __forceinline__ float gs_wave_sum(float v) {
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) v += __shfl_xor(v, o, 64);
    return v;
}

constexpr int GS_T = 64;                                        // tokens per chunk

// ---------------------------------------------------------------- single rows
// A workgroup owns 64 NCOL columns of one head of one segment: lane = column (NCOL of them, 64 apart), the NW waves share the rows.  The first 128 rows of the
// state are on their way from memory while q, k and the decays are made.
template <int NCOL, int GSS_NW>
__global__ __launch_bounds__(64 * GSS_NW) void gated_step_kernel(GatedScanArgs a) {
    extern __shared__ float gs_lds[];
    constexpr int GSS_PRE = 128 / GSS_NW;
    const int D = a.D, VD = a.VD, H = a.H, tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
    float *sq = gs_lds, *sk = sq + D, *sa = sk + D, *sv = sa + D, *red = sv + 64 * NCOL;        // [D], [D], [D], [64 NCOL], [NW][64 NCOL]
    const int seg = blockIdx.x, h = blockIdx.y, row = a.row0 + seg, slot = a.seg_slot[seg], c0 = blockIdx.z * 64 * NCOL;
    float *Sg = a.S + ((size_t)slot * H + h) * (size_t)D * VD + c0 + lane;
    float pre[GSS_PRE][NCOL];
#pragma unroll
    for (int i = 0; i < GSS_PRE; i++) {
        const int d = wave + GSS_NW * i;
#pragma unroll
        for (int j = 0; j < NCOL; j++) pre[i][j] = d < D && c0 + 64 * j + lane < VD ? Sg[(size_t)d * VD + 64 * j] : 0.0f;
    }
    const float *p = a.p + (size_t)row * a.ld_p;
    const int back = a.conv_taps - 1;
    const float *cs = a.conv_wt ? a.conv_state + (size_t)slot * back * a.conv_C : nullptr;
    const auto input = [&](int c) {                             // channel c of the token, convolved where the layer does that
        const float x = p[c];
        if (!a.conv_wt) return x;
        float w[8], u[8];                                       // (taps on their way together)
#pragma unroll
        for (int j = 0; j < 8; j++) { const bool in = j < back; w[j] = in ? a.conv_wt[(size_t)j * a.conv_C + c] : 0.0f; u[j] = in ? cs[(size_t)j * a.conv_C + c] : 0.0f; }
        const float wl = a.conv_wt[(size_t)back * a.conv_C + c];
        float s = a.conv_b ? a.conv_b[c] : 0.0f;
#pragma unroll
        for (int j = 0; j < 8; j++) s = fmaf(w[j], u[j], s);
        for (int j = 8; j < back; j++) s = fmaf(a.conv_wt[(size_t)j * a.conv_C + c], cs[(size_t)j * a.conv_C + c], s);
        return gs_silu(fmaf(wl, x, s));
    };
    float ah = 1.0f, kmul = 1.0f;
    if (a.dt) {                                                 // one decay per head
        kmul = gs_softplus(a.dt[(size_t)row * a.ld_dt + h] + a.dt_bias[h]);
        ah = expf(-expf(a.A_log[h]) * kmul);
    }
    const int qk = (h / a.share) * D, NI = 2 * D + 64 * NCOL;   // query and key entries, value columns: one item per thread at a time
    for (int i = tid; i < NI; i += 64 * GSS_NW) {
        const int d = i < D ? i : i - D, c = i - 2 * D;
        if (c < 0) {
            const bool isq = i < D;
            const float u = input((isq ? a.off_q : a.off_k) + qk + d);
            if (isq) sq[d] = u * a.q_scale; else sk[d] = u * kmul;
        } else sv[c] = c0 + c < VD ? input(a.off_v + h * VD + c0 + c) : 0.0f;
    }
    if (a.dt) for (int d = tid; d < D; d += 64 * GSS_NW) sa[d] = ah;
    else if (!a.lr_w) for (int d = tid; d < D; d += 64 * GSS_NW) sa[d] = a.alpha[(size_t)row * a.ld_alpha + (size_t)h * D + d];
    if (!a.dt && a.lr_w) {                                      // the second half of the low-rank decay: four lanes share a channel's dot product
        const float *z1 = p + a.off_lr;
        for (int d0 = 0; d0 < D; d0 += 16 * GSS_NW) {
            const int d = d0 + (tid >> 2);
            float z = 0.0f;
            if (d < D) {
                const unsigned short *w = a.lr_w + ((size_t)h * D + d) * a.rank;
                for (int r = tid & 3; r < a.rank; r += 4) z = fmaf(__uint_as_float((unsigned)w[r] << 16), z1[r], z);
            }
            z += __shfl_xor(z, 1, 64);
            z += __shfl_xor(z, 2, 64);
            if (d < D && (tid & 3) == 0) sa[d] = expf(-gs_softplus(-(z + a.lr_bias[(size_t)h * D + d])) * a.inv_tau);
        }
    }
    __syncthreads();
    float v[NCOL], num[NCOL];
#pragma unroll
    for (int j = 0; j < NCOL; j++) { v[j] = sv[64 * j + lane]; num[j] = 0.0f; }
    const auto entry = [&](int d, int j, float s0) {
        const float s = fmaf(sa[d], s0, sk[d] * v[j]);
        if (c0 + 64 * j + lane < VD) Sg[(size_t)d * VD + 64 * j] = s;
        num[j] = fmaf(s, sq[d], num[j]);
    };
#pragma unroll
    for (int i = 0; i < GSS_PRE; i++) {
        const int d = wave + GSS_NW * i;
        if (d >= D) break;
#pragma unroll
        for (int j = 0; j < NCOL; j++) entry(d, j, pre[i][j]);
    }
#pragma unroll 4
    for (int d = wave + GSS_NW * GSS_PRE; d < D; d += GSS_NW)
#pragma unroll
        for (int j = 0; j < NCOL; j++) entry(d, j, c0 + 64 * j + lane < VD ? Sg[(size_t)d * VD + 64 * j] : 0.0f);
#pragma unroll
    for (int j = 0; j < NCOL; j++) red[wave * 64 * NCOL + 64 * j + lane] = num[j];
    __syncthreads();
    float o = 0.0f;
    const bool mine = tid < 64 * NCOL && c0 + tid < VD;
    if (mine) {
#pragma unroll
        for (int w = 0; w < GSS_NW; w++) o += red[w * 64 * NCOL + tid];
        if (a.skip) o = fmaf(a.skip[h], sv[tid], o);
    }
    if (!a.y) {
        if (mine) a.o[(size_t)row * a.ld_o + (size_t)h * VD + c0 + tid] = o;
        return;
    }
    // the head's unit norm, its weight and the gate (all of the head's columns are here)
    const float gate = mine ? a.gate[(size_t)row * a.ld_gate + (size_t)h * VD + tid] : 0.0f;
    const float ss = gs_wave_sum(o * o);
    __syncthreads();
    if (lane == 0) red[wave] = ss;
    __syncthreads();
    float tot = 0.0f;
#pragma unroll
    for (int w = 0; w < NCOL; w++) tot += red[w];
    if (mine) a.y[(size_t)row * a.ld_y + (size_t)h * VD + tid] = o * (1.0f / sqrtf(tot / (float)VD + a.eps)) * a.norm_w[tid] * gs_silu(gate);
}

// ---------------------------------------------------------------- chunks
// the decays of a batch: alpha[t][n] = sigmoid(sum_r w[n][r] z1[t][r] + bias[n])^inv_tau; thread = channel, eight tokens at a time, the low-rank row in pieces of 32
constexpr int GSD_T = 8, GSD_R = 32;
__global__ __launch_bounds__(256) void gated_decay_kernel(const float *z1, int ld_z, int T, int rank, const unsigned short *w, const float *bias, float inv_tau, int N, float *alpha, int ld_a) {
    __shared__ float sz[GSD_T][GSD_R];
    const int t0 = blockIdx.x * GSD_T, n = blockIdx.y * 256 + threadIdx.x, tid = threadIdx.x;
    const unsigned short *wn = w + (size_t)(n < N ? n : N - 1) * rank;
    float acc[GSD_T];
#pragma unroll
    for (int t = 0; t < GSD_T; t++) acc[t] = 0.0f;
    for (int r0 = 0; r0 < rank; r0 += GSD_R) {
        const int nr = rank - r0 < GSD_R ? rank - r0 : GSD_R;
        unsigned short u[GSD_R];
#pragma unroll
        for (int r = 0; r < GSD_R; r++) u[r] = r < nr ? wn[r0 + r] : 0;
        if (r0 > 0) __syncthreads();
        {
            const int t = tid >> 5, r = tid & 31;
            sz[t][r] = t0 + t < T && r < nr ? z1[(size_t)(t0 + t) * ld_z + r0 + r] : 0.0f;
        }
        __syncthreads();
#pragma unroll
        for (int r = 0; r < GSD_R; r++) {
            const float wr = __uint_as_float((unsigned)u[r] << 16);
#pragma unroll
            for (int t = 0; t < GSD_T; t++) acc[t] = fmaf(wr, sz[t][r], acc[t]);
        }
    }
    if (n >= N) return;
    const float b = bias[n];
#pragma unroll
    for (int t = 0; t < GSD_T; t++)
        if (t0 + t < T) alpha[(size_t)(t0 + t) * ld_a + n] = expf(-gs_softplus(-(acc[t] + b)) * inv_tau);
}

// place of a chunk among all chunks of the launch: no two chunks share one, and rows / 64 + segments places hold them all
__device__ __forceinline__ int gs_chunk_at(const GatedScanArgs &a, int seg, int row0) { return ((row0 - a.row0) >> 6) + seg; }

// decays per key channel: a workgroup makes the 16 rows [16 I, + 16) of A of one chunk of one head, q P of those rows and the scaled k of those rows (I = blockIdx.z).
// Lane = key row s, the four waves share the channels of a slice; a key's running product walks down the rows.
constexpr int GSI_DC = 32, GSI_LD = GSI_DC + 4;
__global__ __launch_bounds__(256) void gated_intra_channel_kernel(GatedScanArgs a, int chunks) {
    __shared__ __attribute__((aligned(16))) float sa[GS_T][GSI_LD], sk[GS_T][GSI_LD], skr[GS_T][GSI_LD], sq[16][GSI_LD], sp[16][GSI_LD];
    __shared__ float G[4][GSI_DC];
    __shared__ float part[4][16][GS_T];
    const int seg = blockIdx.x / chunks, c = blockIdx.x - seg * chunks, h = blockIdx.y, I = blockIdx.z, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const int H = a.H, D = a.D, len = a.seg_len[seg] - c * GS_T, row0 = a.seg_start[seg] + c * GS_T;
    const int nc = len < GS_T ? len : GS_T;
    if (nc <= 16 * I) return;                                   // (uniform: before any barrier)
    const float *q = a.p + a.off_q + (size_t)(h / a.share) * D, *k = a.p + a.off_k + (size_t)(h / a.share) * D, *al = a.alpha + (size_t)h * D;
    float *qh = a.w_q + (size_t)h * D, *kh = a.w_k + (size_t)h * D, *gd = a.w_g + ((size_t)gs_chunk_at(a, seg, row0) * H + h) * D;
    const int J = lane >> 4, diag = J == I ? (lane & 15) : -1;  // key row `lane` sits in block J; in the diagonal block it joins at its own row
    float acc[16];
#pragma unroll
    for (int t = 0; t < 16; t++) acc[t] = 0.0f;
    // a slice's inputs travel memory -> registers -> LDS: the next slice's are on their way while this one is worked on
    float ra[8], rk[8], rq[2];
    const auto request = [&](int dc) {
#pragma unroll
        for (int i = 0; i < 8; i++) {
            const int idx = tid + 256 * i, t = idx >> 5, d = idx & 31;
            const bool in = t < nc && dc + d < D;
            ra[i] = in ? al[(size_t)(row0 + t) * a.ld_alpha + dc + d] : 1.0f;        // (rows past the end: nothing fades, nothing is written)
            rk[i] = in ? k[(size_t)(row0 + t) * a.ld_p + dc + d] : 0.0f;
        }
#pragma unroll
        for (int i = 0; i < 2; i++) {
            const int idx = tid + 256 * i, t = idx >> 5, d = idx & 31;
            rq[i] = 16 * I + t < nc && dc + d < D ? q[(size_t)(row0 + 16 * I + t) * a.ld_p + dc + d] * a.q_scale : 0.0f;
        }
    };
    request(0);
    for (int dc = 0; dc < D; dc += GSI_DC) {
        __syncthreads();                                        // (the previous slice has been used up)
#pragma unroll
        for (int i = 0; i < 8; i++) { const int idx = tid + 256 * i; sa[idx >> 5][idx & 31] = ra[i]; sk[idx >> 5][idx & 31] = rk[i]; }
#pragma unroll
        for (int i = 0; i < 2; i++) { const int idx = tid + 256 * i; sq[idx >> 5][idx & 31] = rq[i]; }
        __syncthreads();
        if (dc + GSI_DC < D) request(dc + GSI_DC);
        if (tid < 128) {                                        // keys times the decays behind them inside their block; a block's whole product
            const int d = tid & 31, b = tid >> 5;
            float r = 1.0f;
#pragma unroll
            for (int t = 15; t >= 0; t--) { skr[16 * b + t][d] = sk[16 * b + t][d] * r; r *= sa[16 * b + t][d]; }
            G[b][d] = r;
        } else if (tid < 160) {                                 // beside them: the decays up to every row of this workgroup's block
            const int d = tid & 31;
            float r = 1.0f;
#pragma unroll
            for (int t = 0; t < 16; t++) { r *= sa[16 * I + t][d]; sp[t][d] = r; }
        }
        __syncthreads();
#pragma unroll
        for (int i = 0; i < 2; i++) {
            const int d = tid & 31, t = (tid >> 5) + 8 * i, row = 16 * I + t;
            if (row < nc && dc + d < D) {
                float pf = sp[t][d], sf = 1.0f;
#pragma unroll
                for (int b = 0; b < 4; b++) { const float g = G[b][d]; if (b < I) pf *= g; else if (b > I) sf *= g; }
                qh[(size_t)(row0 + row) * ((size_t)H * D) + dc + d] = sq[t][d] * pf;
                kh[(size_t)(row0 + row) * ((size_t)H * D) + dc + d] = skr[row][d] * sf;
            }
        }
        if (I == 0 && tid < GSI_DC && dc + tid < D) gd[dc + tid] = (G[0][tid] * G[1][tid]) * (G[2][tid] * G[3][tid]);
#pragma unroll
        for (int g = 0; g < 2; g++) {
            const int d = 8 * wave + 4 * g;
            const f32x4 kr = *reinterpret_cast<const f32x4 *>(&skr[lane][d]), kk = *reinterpret_cast<const f32x4 *>(&sk[lane][d]);
            f32x4 w = J < I ? kr : f32x4{0.0f, 0.0f, 0.0f, 0.0f};
            for (int b = 1; b < I; b++) {                       // the blocks between the key's and the row's
                const f32x4 gb = *reinterpret_cast<const f32x4 *>(&G[b][d]);
                if (b > J) w *= gb;
            }
#pragma unroll
            for (int t = 0; t < 16; t++) {
                const f32x4 a4 = *reinterpret_cast<const f32x4 *>(&sa[16 * I + t][d]), q4 = *reinterpret_cast<const f32x4 *>(&sq[t][d]);
                const bool joins = diag == t;
#pragma unroll
                for (int e = 0; e < 4; e++) {
                    w[e] = joins ? kk[e] : w[e] * a4[e];
                    acc[t] = fmaf(w[e], q4[e], acc[t]);
                }
            }
        }
    }
#pragma unroll
    for (int t = 0; t < 16; t++) part[wave][t][lane] = acc[t];
    __syncthreads();
#pragma unroll
    for (int i = 0; i < 4; i++) {
        const int t = wave + 4 * i, row = 16 * I + t;
        if (row < nc && lane < 16 * (I + 1))
            a.w_A[((size_t)(row0 + row) * H + h) * GS_T + lane] = (part[0][t][lane] + part[1][t][lane]) + (part[2][t][lane] + part[3][t][lane]);
    }
}

// four consecutive entries of a row of n
template <bool VEC>
__device__ __forceinline__ f32x4 gs_load4(const float *row, int d, int n) {
    if (VEC) return d < n ? *reinterpret_cast<const f32x4 *>(row + d) : f32x4{0.0f, 0.0f, 0.0f, 0.0f};
    f32x4 o;
#pragma unroll
    for (int e = 0; e < 4; e++) o[e] = d + e < n ? row[d + e] : 0.0f;
    return o;
}

// one decay per head: A of one chunk of one head (a wave per 16 rows), the factors of every row - w_p[t] = q_scale a_1 .. a_t, w_s[s] = dt_s a_(s+1) .. a_end - and of the chunk
template <bool VEC>
__global__ __launch_bounds__(256) void gated_intra_head_kernel(GatedScanArgs a, int chunks) {
    __shared__ __attribute__((aligned(16))) float sa[GS_T], sdt[GS_T];
    __shared__ float wt[GS_T][GS_T + 1];
    const int seg = blockIdx.x / chunks, c = blockIdx.x - seg * chunks, h = blockIdx.y, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, l16 = lane & 15, lg = lane >> 4;
    const int H = a.H, D = a.D, len = a.seg_len[seg] - c * GS_T, row0 = a.seg_start[seg] + c * GS_T;
    if (len <= 0) return;                                       // (uniform: before the barrier)
    const int nc = len < GS_T ? len : GS_T;
    if (tid < GS_T) {
        float dt = 0.0f, al = 1.0f;                             // (rows past the end: nothing fades, nothing is written)
        if (tid < nc) {
            dt = gs_softplus(a.dt[(size_t)(row0 + tid) * a.ld_dt + h] + a.dt_bias[h]);
            al = expf(-expf(a.A_log[h]) * dt);
        }
        sa[tid] = al; sdt[tid] = dt;
    }
    const int t = 16 * wave + l16;
    const float *q = a.p + (size_t)(row0 + (t < nc ? t : nc - 1)) * a.ld_p + a.off_q + (size_t)(h / a.share) * D;
    const float *k[4];
    f32x4 acc[4];
#pragma unroll
    for (int u = 0; u < 4; u++) {
        const int s = 16 * u + l16;
        k[u] = a.p + (size_t)(row0 + (s < nc ? s : nc - 1)) * a.ld_p + a.off_k + (size_t)(h / a.share) * D;
        acc[u] = f32x4{0.0f, 0.0f, 0.0f, 0.0f};
    }
    for (int d0 = 0; d0 < D; d0 += 16) {
        const int d = d0 + 4 * lg;
        const f32x4 q4 = gs_load4<VEC>(q, d, D);
        f32x4 k4[4];
#pragma unroll
        for (int u = 0; u < 4; u++) k4[u] = gs_load4<VEC>(k[u], d, D);
#pragma unroll
        for (int u = 0; u < 4; u++) {
            if (u > wave) continue;
#pragma unroll
            for (int e = 0; e < 4; e++) acc[u] = __builtin_amdgcn_mfma_f32_16x16x4f32(k4[u][e], q4[e], acc[u], 0, 0, 0);
        }
    }
    __syncthreads();
    {
        // lane = key row: its factor walks down the rows, each wave keeps its own 16; the last wave's final product is what the key still counts at the chunk's end
        float w = 0.0f;
        const float by = sdt[lane] * a.q_scale;
#pragma unroll 4
        for (int u4 = 0; u4 < 4 * wave + 4; u4++) {
            const f32x4 a4 = *reinterpret_cast<const f32x4 *>(&sa[4 * u4]);
#pragma unroll
            for (int e = 0; e < 4; e++) {
                w = 4 * u4 + e == lane ? 1.0f : w * a4[e];
                if (u4 >= 4 * wave) wt[4 * u4 + e][lane] = w * by;
            }
        }
        if (wave == 3 && lane < nc) a.w_s[(size_t)(row0 + lane) * H + h] = w * sdt[lane];
        if (wave == 0) {
            float p = 1.0f;
#pragma unroll 4
            for (int u4 = 0; u4 < GS_T / 4; u4++) {
                const f32x4 a4 = *reinterpret_cast<const f32x4 *>(&sa[4 * u4]);
#pragma unroll
                for (int e = 0; e < 4; e++) p *= 4 * u4 + e <= lane ? a4[e] : 1.0f;
            }
            if (lane < nc) a.w_p[(size_t)(row0 + lane) * H + h] = p * a.q_scale;
            if (lane == GS_T - 1) a.w_g[(size_t)gs_chunk_at(a, seg, row0) * H + h] = p;
        }
    }
    __syncthreads();
    if (t >= nc) return;
    float *A = a.w_A + ((size_t)(row0 + t) * H + h) * GS_T;
#pragma unroll
    for (int u = 0; u < 4; u++) {
        if (u > wave) continue;
        f32x4 o;
#pragma unroll
        for (int r = 0; r < 4; r++) { const int s = 16 * u + 4 * lg + r; o[r] = s <= t ? wt[t][s] * acc[u][r] : 0.0f; }
        *reinterpret_cast<f32x4 *>(A + 16 * u + 4 * lg) = o;
    }
}

// what one chunk adds to the state: sum_s (k_s a_(s+1) .. a_end) v_s^T; a wave makes 32 rows x 16 columns of it (lane = column l & 15, register r of tile i = row
// 16 i + 4 (l >> 4) + r).  No wave waits for another.
template <bool PERCH>
__global__ __launch_bounds__(256) void gated_update_kernel(GatedScanArgs a, int chunks, int CB) {
    const int seg = blockIdx.x / chunks, c = blockIdx.x - seg * chunks, h = blockIdx.y, lane = threadIdx.x & 63, wave = threadIdx.x >> 6, l16 = lane & 15, lg = lane >> 4;
    const int H = a.H, D = a.D, VD = a.VD, d0 = ((int)blockIdx.z / CB) * 32, col = ((int)blockIdx.z % CB) * 64 + 16 * wave + l16;
    const int len = a.seg_len[seg] - c * GS_T, row0 = a.seg_start[seg] + c * GS_T;
    if (len <= 0) return;
    const int nc = len < GS_T ? len : GS_T;
    const bool cin = col < VD;
    const float *kb = PERCH ? a.w_k + (size_t)h * D : a.p + a.off_k + (size_t)(h / a.share) * D;
    const int ld_k = PERCH ? H * D : a.ld_p;
    const float *vb = a.p + a.off_v + (size_t)h * VD + col;
    float k[2][16], v[16];
#pragma unroll
    for (int j = 0; j < 16; j++) {
        const int s = 16 * (j >> 2) + 4 * lg + (j & 3), row = row0 + (s < nc ? s : nc - 1);
#pragma unroll
        for (int i = 0; i < 2; i++) { const int d = d0 + 16 * i + l16; k[i][j] = d < D ? kb[(size_t)row * ld_k + d] : 0.0f; }
        v[j] = s < nc && cin ? vb[(size_t)row * a.ld_p] : 0.0f;
        if (!PERCH) v[j] *= a.w_s[(size_t)row * H + h];
    }
    f32x4 U[2] = {{0.0f, 0.0f, 0.0f, 0.0f}, {0.0f, 0.0f, 0.0f, 0.0f}};
#pragma unroll
    for (int j = 0; j < 16; j++)
#pragma unroll
        for (int i = 0; i < 2; i++) U[i] = __builtin_amdgcn_mfma_f32_16x16x4f32(k[i][j], v[j], U[i], 0, 0, 0);
    float *Uc = a.w_S + ((size_t)gs_chunk_at(a, seg, row0) * H + h) * (size_t)D * VD + col;
#pragma unroll
    for (int i = 0; i < 2; i++)
#pragma unroll
        for (int r = 0; r < 4; r++) { const int d = d0 + 16 * i + 4 * lg + r; if (cin && d < D) Uc[(size_t)d * VD] = U[i][r]; }
}

// the walk over a segment's chunks, one entry of the state per thread: S <- g S + (what the chunk adds), the state in front of the chunk takes the addition's place
constexpr int GSC_AHEAD = 8;
template <bool PERCH>
__global__ __launch_bounds__(256) void gated_carry_kernel(GatedScanArgs a) {
    const int seg = blockIdx.x, h = blockIdx.y, e = (int)blockIdx.z * 256 + (int)threadIdx.x, H = a.H, D = a.D, VD = a.VD;
    if (e >= D * VD) return;
    const int start = a.seg_start[seg], len = a.seg_len[seg], n = (len + GS_T - 1) / GS_T, at0 = gs_chunk_at(a, seg, start);   // (a segment's chunks lie side by side)
    float *Sg = a.S + ((size_t)a.seg_slot[seg] * H + h) * (size_t)D * VD + e;
    float *U = a.w_S + ((size_t)at0 * H + h) * (size_t)D * VD + e;
    const float *g = PERCH ? a.w_g + ((size_t)at0 * H + h) * D + e / VD : a.w_g + (size_t)at0 * H + h;
    const size_t us = (size_t)H * D * VD, gs = PERCH ? (size_t)H * D : (size_t)H;
    float S = *Sg;
    for (int c0 = 0; c0 < n; c0 += GSC_AHEAD) {
        float u[GSC_AHEAD], f[GSC_AHEAD];
#pragma unroll
        for (int i = 0; i < GSC_AHEAD; i++)
            if (c0 + i < n) { u[i] = U[(size_t)(c0 + i) * us]; f[i] = g[(size_t)(c0 + i) * gs]; }
#pragma unroll
        for (int i = 0; i < GSC_AHEAD; i++)
            if (c0 + i < n) { U[(size_t)(c0 + i) * us] = S; S = fmaf(f[i], S, u[i]); }
    }
    *Sg = S;
}

// the outputs of 64 columns of one chunk of one head: (q P) S_0 + A V (+ skip v); a wave per 16 tokens, S_0 and V through LDS
template <bool PERCH, bool VEC>
__global__ __launch_bounds__(256) void gated_out_kernel(GatedScanArgs a, int chunks) {
    constexpr int LD = 68;
    __shared__ float sS[GS_T][LD], sV[GS_T][LD];
    const int seg = blockIdx.x / chunks, c = blockIdx.x - seg * chunks, h = blockIdx.y, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, l16 = lane & 15, lg = lane >> 4;
    const int H = a.H, D = a.D, VD = a.VD, len = a.seg_len[seg] - c * GS_T, row0 = a.seg_start[seg] + c * GS_T, col = blockIdx.z * 64 + lane;
    if (len <= 0) return;                                       // (uniform: before any barrier)
    const int nc = len < GS_T ? len : GS_T;
    const float *Sc = a.w_S + ((size_t)gs_chunk_at(a, seg, row0) * H + h) * (size_t)D * VD;
    const int t = 16 * wave + l16, tr = row0 + (t < nc ? t : nc - 1);
    const float *q = PERCH ? a.w_q + ((size_t)tr * H + h) * D : a.p + (size_t)tr * a.ld_p + a.off_q + (size_t)(h / a.share) * D;
    const float *A = a.w_A + ((size_t)tr * H + h) * GS_T;
    float nv[16], ns[16];
    f32x4 A4[4], acc[4], q4[4];
    const auto request = [&](int ds) {
#pragma unroll
        for (int u = 0; u < 4; u++) q4[u] = gs_load4<VEC>(q, ds + 16 * u + 4 * lg, D);
#pragma unroll
        for (int i = 0; i < 16; i++) { const int d = ds + wave + 4 * i; ns[i] = d < D && col < VD ? Sc[(size_t)d * VD + col] : 0.0f; }
    };
    request(0);                                                 // (everything the first products need is on its way before any of it is waited for)
#pragma unroll
    for (int i = 0; i < 16; i++) { const int s = wave + 4 * i; nv[i] = s < nc && col < VD ? a.p[(size_t)(row0 + s) * a.ld_p + a.off_v + (size_t)h * VD + col] : 0.0f; }
#pragma unroll
    for (int u = 0; u < 4; u++) {
        A4[u] = u <= wave ? *reinterpret_cast<const f32x4 *>(A + 16 * u + 4 * lg) : f32x4{0.0f, 0.0f, 0.0f, 0.0f};
        acc[u] = f32x4{0.0f, 0.0f, 0.0f, 0.0f};
    }
#pragma unroll
    for (int i = 0; i < 16; i++) sV[wave + 4 * i][lane] = nv[i];
    for (int ds = 0; ds < D; ds += GS_T) {
        if (ds > 0) __syncthreads();                            // (the previous slice has been used up)
        f32x4 qs[4];
#pragma unroll
        for (int u = 0; u < 4; u++) qs[u] = q4[u];
#pragma unroll
        for (int i = 0; i < 16; i++) sS[wave + 4 * i][lane] = ns[i];
        __syncthreads();
        if (ds + GS_T < D) request(ds + GS_T);
#pragma unroll
        for (int u = 0; u < 4; u++)
#pragma unroll
            for (int e = 0; e < 4; e++)
#pragma unroll
                for (int ct = 0; ct < 4; ct++) acc[ct] = __builtin_amdgcn_mfma_f32_16x16x4f32(qs[u][e], sS[16 * u + 4 * lg + e][16 * ct + l16], acc[ct], 0, 0, 0);
    }
    if (!PERCH) {
        f32x4 w;
#pragma unroll
        for (int r = 0; r < 4; r++) { const int tt = 16 * wave + 4 * lg + r; w[r] = a.w_p[(size_t)(row0 + (tt < nc ? tt : nc - 1)) * H + h]; }
#pragma unroll
        for (int ct = 0; ct < 4; ct++) acc[ct] *= w;
    }
#pragma unroll
    for (int u = 0; u < 4; u++) {
        if (u > wave) continue;
#pragma unroll
        for (int e = 0; e < 4; e++)
#pragma unroll
            for (int ct = 0; ct < 4; ct++) acc[ct] = __builtin_amdgcn_mfma_f32_16x16x4f32(A4[u][e], sV[16 * u + 4 * lg + e][16 * ct + l16], acc[ct], 0, 0, 0);
    }
    const float skip = a.skip ? a.skip[h] : 0.0f;
#pragma unroll
    for (int ct = 0; ct < 4; ct++)
#pragma unroll
        for (int r = 0; r < 4; r++) {
            const int tt = 16 * wave + 4 * lg + r, cc = 16 * ct + l16;
            if (tt < nc && (int)blockIdx.z * 64 + cc < VD)
                a.o[(size_t)(row0 + tt) * a.ld_o + (size_t)h * VD + blockIdx.z * 64 + cc] = a.skip ? fmaf(skip, sV[tt][cc], acc[ct][r]) : acc[ct][r];
        }
}

// y[t][c] = silu(bias[c] + sum_j wt[j][c] u_(t - taps + 1 + j)[c]); inputs in front of a segment's first row come from the slot
template <bool VEC>
__global__ __launch_bounds__(256) void conv_silu_kernel(const float *p, int ld_p, int C, const float *wt, const float *bias, int taps, const float *state, const int32_t *tok_ago,
                                                        const int32_t *tok_slot, float *y, int ld_y) {
    const int t = blockIdx.x, back = taps - 1, ago = tok_ago[t];
    const float *st = state ? state + (size_t)tok_slot[t] * back * C : nullptr;
    if (VEC) {
        const int c = 4 * ((int)blockIdx.y * 256 + (int)threadIdx.x);
        if (c >= C) return;
        f32x4 s = bias ? *reinterpret_cast<const f32x4 *>(bias + c) : f32x4{0.0f, 0.0f, 0.0f, 0.0f};
#pragma unroll 4
        for (int j = 0; j <= back; j++) {
            const int b = back - j;
            const f32x4 w = *reinterpret_cast<const f32x4 *>(wt + (size_t)j * C + c);
            const f32x4 u = *reinterpret_cast<const f32x4 *>(b <= ago ? p + (size_t)(t - b) * ld_p + c : st + (size_t)(back - (b - ago)) * C + c);
#pragma unroll
            for (int e = 0; e < 4; e++) s[e] = fmaf(w[e], u[e], s[e]);
        }
#pragma unroll
        for (int e = 0; e < 4; e++) s[e] = gs_silu(s[e]);
        *reinterpret_cast<f32x4 *>(y + (size_t)t * ld_y + c) = s;
    } else {
        const int c = (int)blockIdx.y * 256 + (int)threadIdx.x;
        if (c >= C) return;
        float s = bias ? bias[c] : 0.0f;
        for (int j = 0; j <= back; j++) {
            const int b = back - j;
            s = fmaf(wt[(size_t)j * C + c], b <= ago ? p[(size_t)(t - b) * ld_p + c] : st[(size_t)(back - (b - ago)) * C + c], s);
        }
        y[(size_t)t * ld_y + c] = gs_silu(s);
    }
}

// y = o silu(z), every one of `parts` equal parts of the row over its root mean square, times w.  mv.state set (every row is a segment of its own): the launch also
// moves the convolution inputs on - nobody reads them any more
__global__ __launch_bounds__(256) void gated_norm_kernel(const float *o, int ld_o, const float *z, int ld_z, const float *w, int parts, int n, float eps, float *y, int ld_y,
                                                         ConvMove mv) {
    __shared__ float sh[4];
    const int t = blockIdx.x, part = blockIdx.y, tid = threadIdx.x;
    if (part >= parts) {                                        // (the launch's further workgroups: a channel per thread)
        const int c = (part - parts) * 256 + tid, back = mv.taps - 1;
        if (c >= mv.C) return;
        float *st = mv.state + (size_t)mv.seg_slot[t] * back * mv.C + c;
        const float u = mv.p[(size_t)t * mv.ld_p + c];
        float keep[8];
#pragma unroll
        for (int j = 0; j < 8; j++) keep[j] = j + 1 < back ? st[(size_t)(j + 1) * mv.C] : 0.0f;
#pragma unroll
        for (int j = 0; j < 8; j++) if (j + 1 < back) st[(size_t)j * mv.C] = keep[j];
        for (int j = 8; j + 1 < back; j++) st[(size_t)j * mv.C] = st[(size_t)(j + 1) * mv.C];
        st[(size_t)(back - 1) * mv.C] = u;
        return;
    }
    const float *orow = o + (size_t)t * ld_o + (size_t)part * n, *zr = z + (size_t)t * ld_z + (size_t)part * n;
    float keep[8], ss = 0.0f;
#pragma unroll
    for (int i = 0; i < 8; i++) {
        const int c = tid + 256 * i;
        keep[i] = c < n ? orow[c] * gs_silu(zr[c]) : 0.0f;
        ss = fmaf(keep[i], keep[i], ss);
    }
    for (int c = tid + 2048; c < n; c += 256) { const float v = orow[c] * gs_silu(zr[c]); ss = fmaf(v, v, ss); }
    ss = gs_wave_sum(ss);
    if ((tid & 63) == 0) sh[tid >> 6] = ss;
    __syncthreads();
    const float inv = 1.0f / sqrtf(((sh[0] + sh[1]) + (sh[2] + sh[3])) / (float)n + eps);
    float *yr = y + (size_t)t * ld_y + (size_t)part * n;
    const float *wr = w + (size_t)part * n;
#pragma unroll
    for (int i = 0; i < 8; i++) { const int c = tid + 256 * i; if (c < n) yr[c] = keep[i] * inv * wr[c]; }
    for (int c = tid + 2048; c < n; c += 256) yr[c] = orow[c] * gs_silu(zr[c]) * inv * wr[c];
}

template <int NCOL>
static hipError_t launch_gated_step(const GatedScanArgs &a, int nz, hipStream_t st) {
    const int nw = a.D >= 64 ? 16 : 8;                          // (a head's state is read by one workgroup: the more waves, the more of it is on its way)
    const size_t lds = ((size_t)3 * a.D + 64 * NCOL + (size_t)nw * 64 * NCOL) * sizeof(float);
    const dim3 grid((unsigned)a.n_seg, (unsigned)a.H, (unsigned)nz);
    if (nw == 16) hipLaunchKernelGGL((gated_step_kernel<NCOL, 16>), grid, dim3(1024), lds, st, a);
    else hipLaunchKernelGGL((gated_step_kernel<NCOL, 8>), grid, dim3(512), lds, st, a);
    return hipGetLastError();
}

}  // namespace

bool gated_scan_shape_ok(int H, int share, int D, int VD) { return H >= 1 && share >= 1 && H % share == 0 && D >= 1 && D <= GATED_SCAN_MAX_DIM && VD >= 1; }
bool gated_step_closes(int VD) { return VD <= 256; }

hipError_t launch_gated_scan(const GatedScanArgs &a, hipStream_t st) {
    if (a.n_seg <= 0 || a.max_len <= 0) return hipSuccess;
    const bool perch = a.dt == nullptr;
    if (!gated_scan_shape_ok(a.H, a.share, a.D, a.VD) || !a.p || !a.S || (!perch && (!a.dt_bias || !a.A_log))) return hipErrorInvalidValue;
    if (a.max_len == 1) {
        if ((perch && !a.lr_w && !a.alpha) || (a.lr_w && !a.lr_bias) || (a.conv_wt && a.conv_taps > 1 && !a.conv_state) || (!a.y && !a.o)) return hipErrorInvalidValue;
        if (a.y) {
            if (!gated_step_closes(a.VD) || !a.gate || !a.norm_w) return hipErrorInvalidValue;
            if (a.VD <= 64) return launch_gated_step<1>(a, 1, st);
            if (a.VD <= 128) return launch_gated_step<2>(a, 1, st);
            return launch_gated_step<4>(a, 1, st);
        }
        return launch_gated_step<1>(a, (a.VD + 63) / 64, st);
    }
    if ((perch && (!a.alpha || !a.w_q || !a.w_k)) || (!perch && (!a.w_p || !a.w_s)) || !a.w_A || !a.w_g || !a.w_S || !a.o) return hipErrorInvalidValue;
    const int chunks = (a.max_len + GS_T - 1) / GS_T, CB = (a.VD + 63) / 64, DB = (a.D + 31) / 32, EB = (int)(((long long)a.D * a.VD + 255) / 256);
    const auto al16 = [](const void *p) { return (reinterpret_cast<uintptr_t>(p) & 15) == 0; };
    const dim3 ic((unsigned)(a.n_seg * chunks), (unsigned)a.H), ug(ic.x, ic.y, (unsigned)(DB * CB)), cg((unsigned)a.n_seg, (unsigned)a.H, (unsigned)EB), og((unsigned)(a.n_seg * chunks), (unsigned)a.H, (unsigned)CB);
    if (perch) {
        const bool vec = (a.D & 3) == 0 && al16(a.w_q);
        hipLaunchKernelGGL(gated_intra_channel_kernel, dim3(ic.x, ic.y, 4), dim3(256), 0, st, a, chunks);
        hipLaunchKernelGGL(gated_update_kernel<true>, ug, dim3(256), 0, st, a, chunks, CB);
        hipLaunchKernelGGL(gated_carry_kernel<true>, cg, dim3(256), 0, st, a);
        if (vec) hipLaunchKernelGGL((gated_out_kernel<true, true>), og, dim3(256), 0, st, a, chunks);
        else hipLaunchKernelGGL((gated_out_kernel<true, false>), og, dim3(256), 0, st, a, chunks);
        return hipGetLastError();
    }
    const bool vec = ((a.D | a.ld_p | a.off_q | a.off_k) & 3) == 0 && al16(a.p);
    if (vec) hipLaunchKernelGGL(gated_intra_head_kernel<true>, ic, dim3(256), 0, st, a, chunks);
    else hipLaunchKernelGGL(gated_intra_head_kernel<false>, ic, dim3(256), 0, st, a, chunks);
    hipLaunchKernelGGL(gated_update_kernel<false>, ug, dim3(256), 0, st, a, chunks, CB);
    hipLaunchKernelGGL(gated_carry_kernel<false>, cg, dim3(256), 0, st, a);
    if (vec) hipLaunchKernelGGL((gated_out_kernel<false, true>), og, dim3(256), 0, st, a, chunks);
    else hipLaunchKernelGGL((gated_out_kernel<false, false>), og, dim3(256), 0, st, a, chunks);
    return hipGetLastError();
}

hipError_t launch_gated_decay(const float *z1, int ld_z, int T, int rank, const unsigned short *w, const float *bias, float inv_tau, int N, float *alpha, int ld_a, hipStream_t st) {
    if (T <= 0 || N <= 0) return hipSuccess;
    if (rank < 1 || !z1 || !w || !bias || !alpha) return hipErrorInvalidValue;
    hipLaunchKernelGGL(gated_decay_kernel, dim3((unsigned)((T + GSD_T - 1) / GSD_T), (unsigned)((N + 255) / 256)), dim3(256), 0, st, z1, ld_z, T, rank, w, bias, inv_tau, N, alpha, ld_a);
    return hipGetLastError();
}

hipError_t launch_conv_silu(const float *p, int ld_p, int C, const float *wt, const float *bias, int taps, const float *state, const int32_t *tok_ago, const int32_t *tok_slot, int T,
                            float *y, int ld_y, hipStream_t st) {
    if (T <= 0 || C <= 0) return hipSuccess;
    if (taps < 1 || !p || !wt || !y || !tok_ago || !tok_slot || (taps > 1 && !state)) return hipErrorInvalidValue;
    const auto al16 = [](const void *q) { return (reinterpret_cast<uintptr_t>(q) & 15) == 0; };
    const bool vec = ((C | ld_p | ld_y) & 3) == 0 && al16(p) && al16(wt) && al16(y) && (!bias || al16(bias)) && (!state || al16(state));
    if (vec) hipLaunchKernelGGL(conv_silu_kernel<true>, dim3((unsigned)T, (unsigned)((C / 4 + 255) / 256)), dim3(256), 0, st, p, ld_p, C, wt, bias, taps, state, tok_ago, tok_slot, y, ld_y);
    else hipLaunchKernelGGL(conv_silu_kernel<false>, dim3((unsigned)T, (unsigned)((C + 255) / 256)), dim3(256), 0, st, p, ld_p, C, wt, bias, taps, state, tok_ago, tok_slot, y, ld_y);
    return hipGetLastError();
}

hipError_t launch_gated_norm(const float *o, int ld_o, const float *z, int ld_z, const float *w, int T, int parts, int n, float eps, float *y, int ld_y, const ConvMove &mv, hipStream_t st) {
    if (T <= 0) return hipSuccess;
    if (parts < 1 || n < 1 || !o || !z || !w || !y || (mv.state && (mv.taps < 2 || mv.C < 1 || !mv.p || !mv.seg_slot))) return hipErrorInvalidValue;
    const unsigned movers = mv.state ? (unsigned)((mv.C + 255) / 256) : 0;
    hipLaunchKernelGGL(gated_norm_kernel, dim3((unsigned)T, (unsigned)parts + movers), dim3(256), 0, st, o, ld_o, z, ld_z, w, parts, n, eps, y, ld_y, mv);
    return hipGetLastError();
}

}  // namespace mi355
