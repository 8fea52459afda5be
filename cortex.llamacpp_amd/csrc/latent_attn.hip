// latent_attn.hip — attention through a low-rank latent, on the cache's latent rows themselves.
//
// A token's cache row is [c | r]: the RMS-normed latent c (kv_rank floats) and one rotated key part r (rot floats) shared by all heads.  With W_uk folded
// into the query (qa = W_uk_h^T q_h, a per-head product of mmb.hip) a head's score against a cell is one dot product of length kv_rank + rot,
//   s = (qa . c + rope(q_rot) . r) * scale,
// and the attended value is the weighted sum of latents, unfolded through W_uv afterwards - keys and values are never materialised, every head reads the
// same row.  Visibility: same sequence, 0 <= pos_query - pos_cell < window (window 0: no limit).  The softmax denominator takes one extra term exp(sink_h),
// a learned per-head logit with neither key nor value behind it.  An optional output gate multiplies head h's attended latent by sigmoid(gate[t][h]) (a factor per
// head: it commutes with W_uv).  Everything here is f32: positions, angles, scores, weights, the running sums.
//
// latent_tile (rows that allow 16-byte loads): (row, head) pairs as the columns of products on the f32 matrix cores; latent_attn: one workgroup per pair, any alignment.
// Scans cut into runs of cells leave records that latent_attn_merge joins.
//
// latent_prep: per token, the two RMS norms behind the down-projections (query latent -> cq, key / value latent -> cache row) and the rotation of the
// shared key part into the cache row.  Interleaved pairs (2i, 2i + 1), or entry i with entry i + half the turning part; the per-pair frequency table (YaRN blend included) comes from the host.
#include "attn_merge_dev.h"
#include "kernels.h"

namespace mi355 {

namespace {

__device__ __forceinline__ float wave_sum(float v) {
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) v += __shfl_xor(v, o, 64);
    return v;
}
__device__ float block_sum_256(float v, float *sh) {
    v = wave_sum(v);
    __syncthreads();
    if ((threadIdx.x & 63) == 0) sh[threadIdx.x >> 6] = v;
    __syncthreads();
    return sh[0] + sh[1] + sh[2] + sh[3];
}

// entry i of the turning part: its pair's index, the places of the pair's two entries, and which of them it is
struct LatentPair { int pr, iu, iv; bool second; };
__device__ __forceinline__ LatentPair latent_pair(int i, int dims, int halves) {
    const int half = dims >> 1;
    if (halves) { const int pr = i < half ? i : i - half; return {pr, pr, pr + half, i >= half}; }
    return {i >> 1, i & ~1, i | 1, (i & 1) != 0};
}
// the factor of head h's attended latent: 1 over the softmax denominator, times the output gate
__device__ __forceinline__ float latent_out_factor(const LatentAttnArgs &a, int t, int h, float den) {
    float inv = den > 0.0f ? 1.0f / den : 0.0f;
    if (a.gate) inv *= 1.0f / (1.0f + expf(-a.gate[(size_t)t * a.ld_gate + h]));
    return inv;
}

__global__ __launch_bounds__(256) void latent_prep_kernel(LatentPrepArgs a) {
    __shared__ float sh[4];
    const int t = blockIdx.x, tid = threadIdx.x;
    const float *row = a.a + (size_t)t * a.ld_a;
    // query latent
    float ss = 0.0f;
    for (int i = tid; i < a.q_rank; i += 256) { const float v = row[i]; ss = fmaf(v, v, ss); }
    ss = block_sum_256(ss, sh);
    float inv = 1.0f / sqrtf(ss / (float)a.q_rank + a.eps);
    for (int i = tid; i < a.q_rank; i += 256) a.cq[(size_t)t * a.q_rank + i] = row[i] * inv * a.wq_norm[i];
    // key / value latent -> cache row
    const float *kv = row + a.q_rank;
    float *dst = a.cache + (size_t)a.tok_cell[t] * (a.kv_rank + a.rot);
    ss = 0.0f;
    for (int i = tid; i < a.kv_rank; i += 256) { const float v = kv[i]; ss = fmaf(v, v, ss); }
    ss = block_sum_256(ss, sh);
    inv = 1.0f / sqrtf(ss / (float)a.kv_rank + a.eps);
    for (int i = tid; i < a.kv_rank; i += 256) dst[i] = kv[i] * inv * a.wkv_norm[i];
    // shared rotated key part
    const float *kr = kv + a.kv_rank;
    const float p = (float)a.tok_pos[t];
    for (int i = tid; i < a.rot; i += 256) {
        if (i < a.rot_dims) {
            const LatentPair q = latent_pair(i, a.rot_dims, a.rot_halves);
            const float ang = p * a.rot_freq[q.pr], c = cosf(ang) * a.rot_mscale, s = sinf(ang) * a.rot_mscale;
            const float u = kr[q.iu], v = kr[q.iv];
            dst[a.kv_rank + i] = q.second ? v * c + u * s : u * c - v * s;
        } else dst[a.kv_rank + i] = kr[i];
    }
}

typedef float f32x4 __attribute__((ext_vector_type(4)));

constexpr int LA_MAX_L = 1088;                                  // kv_rank + rot the attention kernel is instantiated for (17 x 64)

// One workgroup per (token, head), NW waves.  A wave works on four cells at a time: each 16-lane group owns one cell, its lanes hold the row's elements
// 64 j + 4 li .. + 3 (16-byte loads, the whole group reads 256 contiguous bytes per j) and the matching running sums; the next four cells of the wave are
// requested before the current ones are used.  Every group keeps its own running maximum / sum / weighted latent; groups, then waves, are merged at the
// end together with the sink term.  NJ = ceil((kv_rank + rot) / 64); VEC: rows are 16-byte aligned (kv_rank + rot a multiple of 4).
template <int NJ, bool VEC>
__global__ __launch_bounds__(512) void latent_attn_kernel(LatentAttnArgs a) {
    extern __shared__ float lds[];
    const int KR = a.kv_rank, R = a.rot, L = KR + R, LP = NJ * 64;
    const int NW = blockDim.x >> 6;
    float *qv = lds;                                            // [LP] (zero beyond L)
    float *wm = lds + LP, *wl = wm + NW, *wacc = wl + NW;        // [NW], [NW], [NW][LP]
    const int t = blockIdx.x, h = blockIdx.y, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, g = lane >> 4, li = lane & 15;
    const int tpos = a.tok_pos[t];
    const uint64_t sbit = 1ull << (a.tok_seq[t] & 63);
    for (int i = tid; i < LP; i += blockDim.x) {
        float v = 0.0f;
        if (i < KR) v = a.qa[(size_t)t * a.ld_qa + (size_t)h * KR + i];
        else if (i < L) {
            const float *qr = a.q + (size_t)t * a.ld_q + (size_t)h * (a.dim + R) + a.dim;
            const int r = i - KR;
            if (r < a.rot_dims) {
                const LatentPair q = latent_pair(r, a.rot_dims, a.rot_halves);
                const float ang = (float)tpos * a.rot_freq[q.pr], c = cosf(ang) * a.rot_mscale, sn = sinf(ang) * a.rot_mscale;
                const float u = qr[q.iu], w = qr[q.iv];
                v = q.second ? w * c + u * sn : u * c - w * sn;
            } else v = qr[r];
        }
        qv[i] = v;
    }
    __syncthreads();
    float acc[NJ][4], cur[NJ][4], nxt[NJ][4];
#pragma unroll
    for (int j = 0; j < NJ; j++)
#pragma unroll
        for (int e = 0; e < 4; e++) { acc[j][e] = 0.0f; cur[j][e] = 0.0f; nxt[j][e] = 0.0f; }
    float m = -INFINITY, l = 0.0f;
    int n_kv = *a.n_kv_dev;
    if (a.tok_hi) n_kv = a.tok_hi[t] < n_kv ? a.tok_hi[t] : n_kv;
    const int stride = NW * 4;
    // gridDim.z > 1 (single-token steps): the scanned range is cut into that many runs of cells, one workgroup each; the runs' records are merged by
    // latent_attn_merge_kernel
    int c_lo = 0, c_hi = n_kv;
    if (gridDim.z > 1) {
        const int per = ((n_kv + (int)gridDim.z - 1) / (int)gridDim.z + stride - 1) / stride * stride;
        c_lo = (int)blockIdx.z * per;
        c_hi = c_lo + per < n_kv ? c_lo + per : n_kv;
    }
    const auto visible = [&](int c) {
        if (c >= c_hi) return false;
        const int cp = a.cell_pos[c];
        return cp >= 0 && cp <= tpos && (a.cell_seq[c] & sbit) != 0 && !(a.window > 0 && tpos - cp >= a.window);
    };
    const auto fetch = [&](int c, bool vis, float (&dst)[NJ][4]) {
        const float *row = a.cache + (size_t)c * L;
#pragma unroll
        for (int j = 0; j < NJ; j++) {
            const int e0 = 64 * j + 4 * li;
            if (VEC) {
                float4 v = make_float4(0.0f, 0.0f, 0.0f, 0.0f);
                if (vis && e0 < L) v = *reinterpret_cast<const float4 *>(row + e0);
                dst[j][0] = v.x; dst[j][1] = v.y; dst[j][2] = v.z; dst[j][3] = v.w;
            } else {
#pragma unroll
                for (int e = 0; e < 4; e++) dst[j][e] = vis && e0 + e < L ? row[e0 + e] : 0.0f;
            }
        }
    };
    int c = c_lo + wave * 4 + g;
    bool vis = visible(c);
    fetch(c, vis, cur);
    for (int c0 = c_lo; c0 < c_hi; c0 += stride) {              // (uniform trip count: the shuffles below are executed by whole waves)
        const int cn = c + stride;
        const bool visn = visible(cn);
        fetch(cn, visn, nxt);
        float dot = 0.0f;
#pragma unroll
        for (int j = 0; j < NJ; j++) {
            const float4 q4 = *reinterpret_cast<const float4 *>(qv + 64 * j + 4 * li);
            dot = fmaf(cur[j][0], q4.x, dot); dot = fmaf(cur[j][1], q4.y, dot); dot = fmaf(cur[j][2], q4.z, dot); dot = fmaf(cur[j][3], q4.w, dot);
        }
#pragma unroll
        for (int o = 8; o > 0; o >>= 1) dot += __shfl_xor(dot, o, 64);
        if (vis) {
            const float sc = dot * a.scale;
            const float mn = fmaxf(m, sc), alpha = expf(m - mn), p = expf(sc - mn);   // (m = -inf at the group's first cell: alpha = 0)
            l = l * alpha + p;
#pragma unroll
            for (int j = 0; j < NJ; j++)
#pragma unroll
                for (int e = 0; e < 4; e++) acc[j][e] = acc[j][e] * alpha + p * cur[j][e];
            m = mn;
        }
#pragma unroll
        for (int j = 0; j < NJ; j++)
#pragma unroll
            for (int e = 0; e < 4; e++) cur[j][e] = nxt[j][e];
        c = cn; vis = visn;
    }
    // the four groups of a wave -> one record per wave
    float M = fmaxf(m, __shfl_xor(m, 16, 64));
    M = fmaxf(M, __shfl_xor(M, 32, 64));
    const float sg = l > 0.0f ? expf(m - M) : 0.0f;
    l *= sg;
    l += __shfl_xor(l, 16, 64);
    l += __shfl_xor(l, 32, 64);
#pragma unroll
    for (int j = 0; j < NJ; j++)
#pragma unroll
        for (int e = 0; e < 4; e++) {
            float v = acc[j][e] * sg;
            v += __shfl_xor(v, 16, 64);
            v += __shfl_xor(v, 32, 64);
            if (g == 0) wacc[wave * LP + 64 * j + 4 * li + e] = v;
        }
    if (lane == 0) { wm[wave] = M; wl[wave] = l; }
    __syncthreads();
    if (gridDim.z > 1) {                                        // this run's record: maximum, sum, weighted latent (no sink: the merge adds it once)
        float *rec = a.part + (((size_t)t * a.H + h) * gridDim.z + blockIdx.z) * (size_t)(KR + 2);
        float Ms = -INFINITY;
        for (int w = 0; w < NW; w++) if (wl[w] > 0.0f) Ms = fmaxf(Ms, wm[w]);
        float ls = 0.0f;
        for (int w = 0; w < NW; w++) ls += wl[w] > 0.0f ? wl[w] * expf(wm[w] - Ms) : 0.0f;
        if (tid == 0) { rec[0] = Ms; rec[1] = ls; }
        for (int i = tid; i < KR; i += blockDim.x) {
            float o = 0.0f;
            for (int w = 0; w < NW; w++) o += wl[w] > 0.0f ? wacc[w * LP + i] * expf(wm[w] - Ms) : 0.0f;
            rec[2 + i] = o;
        }
        return;
    }
    float MM = a.sink ? a.sink[h] : -INFINITY;
    for (int w = 0; w < NW; w++) MM = fmaxf(MM, wm[w]);
    float den = a.sink ? expf(a.sink[h] - MM) : 0.0f;
    for (int w = 0; w < NW; w++) den += wl[w] > 0.0f ? wl[w] * expf(wm[w] - MM) : 0.0f;
    const float inv = latent_out_factor(a, t, h, den);
    for (int i = tid; i < KR; i += blockDim.x) {
        float o = 0.0f;
        for (int w = 0; w < NW; w++) o += wl[w] > 0.0f ? wacc[w * LP + i] * expf(wm[w] - MM) : 0.0f;
        a.out[(size_t)t * a.ld_out + (size_t)h * KR + i] = o * inv;
    }
}

template <int NT>
__global__ __launch_bounds__(NT) void latent_attn_merge_kernel(LatentAttnArgs a, int splits) {
    __shared__ float fac[ATTN_MERGE_MAX_RUNS], part[NT / 256 * LA_MAX_L], sums[LA_MAX_L];
    const int t = blockIdx.x, h = blockIdx.y, tid = threadIdx.x, KR = a.kv_rank;
    const float den = attn_merge_runs<NT>(a.part + ((size_t)t * a.H + h) * splits * (size_t)(KR + 2), splits, KR, a.sink ? a.sink[h] : -INFINITY, fac, part, sums);
    const float inv = latent_out_factor(a, t, h, den);
    for (int i = tid; i < KR; i += NT) a.out[(size_t)t * a.ld_out + (size_t)h * KR + i] = sums[i] * inv;
}

static hipError_t latent_attn_merge(const LatentAttnArgs &a, int splits, hipStream_t st) {
    if ((long long)a.T * a.H <= ATTN_MERGE_FEW) hipLaunchKernelGGL(latent_attn_merge_kernel<1024>, dim3((unsigned)a.T, (unsigned)a.H), dim3(1024), 0, st, a, splits);
    else hipLaunchKernelGGL(latent_attn_merge_kernel<256>, dim3((unsigned)a.T, (unsigned)a.H), dim3(256), 0, st, a, splits);
    return hipGetLastError();
}

template <int NJ>
static hipError_t launch_latent_attn_nj(const LatentAttnArgs &a, hipStream_t st) {
    // few (token, head) pairs - single-token steps - get eight waves each: more cells in flight where the grid alone cannot fill the device
    const int nw = (long long)a.T * a.H <= 1024 ? 8 : 4;
    const size_t lds = (size_t)(NJ * 64 + 2 * nw + nw * NJ * 64) * sizeof(float);
    const bool vec = ((a.kv_rank + a.rot) & 3) == 0 && (reinterpret_cast<uintptr_t>(a.cache) & 15) == 0;
    const int splits = a.part && (long long)a.T * a.H <= LATENT_ATTN_SPLIT_MAX_PAIRS && (size_t)a.T * a.H * LATENT_ATTN_SPLITS * (a.kv_rank + 2) <= a.part_floats ? LATENT_ATTN_SPLITS : 1;
    const dim3 grid((unsigned)a.T, (unsigned)a.H, (unsigned)splits);
    if (vec) hipLaunchKernelGGL((latent_attn_kernel<NJ, true>), grid, dim3(64 * nw), lds, st, a);
    else hipLaunchKernelGGL((latent_attn_kernel<NJ, false>), grid, dim3(64 * nw), lds, st, a);
    return splits > 1 ? latent_attn_merge(a, splits, st) : hipGetLastError();
}

// ---- the same attention on the f32 matrix cores: every head of every row reads the same cache rows, so (row, head) pairs are the columns of one product.
// One workgroup per (tile of 16 R pairs, run of cells), 8 waves, BC cells per block.  v_mfma_f32_16x16x4_f32 (f32 operands, f32 accumulation): lane l holds
// A[l & 15][l >> 4], B[l >> 4][l & 15], register r of the result is D[4 (l >> 4) + r][l & 15]; the order of k is free as long as A and B agree, so a lane
// loads 4 consecutive floats (16 bytes) and feeds them to 4 products.
//   scores:  A = cache rows (i = cell), B = queries (j = pair; in LDS, turned on the way in): a wave takes 16 cells x 16 pairs; where a block has fewer such
//            pieces than the workgroup waves, KS waves share one piece, each a part of the row's length, and their partial sums meet in the softmax
//   softmax: 16 lanes per pair; weights back to LDS
//   values:  A = cache rows (i = latent entry, k = cell), B = weights (k = cell, j = pair): a wave takes 64 entries x 16 pairs; entry i of tile jj stands for
//            64 J + 4 i + jj, which makes every load 16 bytes and a lane's results 16 neighbouring entries of its pair
constexpr int LT_NW = 8;
constexpr int lt_pieces(int R, int BC) { return (BC / 16) * R; }
constexpr int lt_ks(int R, int BC) { return lt_pieces(R, BC) >= LT_NW ? 1 : LT_NW / lt_pieces(R, BC); }
constexpr size_t lt_lds_floats(int R, int BC, int LQ) { return (size_t)16 * R * (LQ + 4) + (size_t)lt_ks(R, BC) * 16 * R * (BC + 4) + 3 * 16 * R + 4 + 64 * R + 2 * 16 * R; }

// NT: tasks (64 latent entries x 16 pairs) a wave owns at most
template <int R, int BC, int NT>
__global__ __launch_bounds__(64 * LT_NW) void latent_tile_kernel(LatentAttnArgs a, int LQ) {
    constexpr int BQ = 16 * R, LDS_S = BC + 4, KS = lt_ks(R, BC), NS = BC / 16;
    extern __shared__ float lds[];
    const int KR = a.kv_rank, RT = a.rot, L = KR + RT, H = a.H, LDQ = LQ + 4;
    float *Q = lds, *S = Q + (size_t)BQ * LDQ, *ms = S + (size_t)KS * BQ * LDS_S, *ls = ms + BQ, *al = ls + BQ;
    int *red = reinterpret_cast<int *>(al + BQ);
    uint64_t *vmask2 = reinterpret_cast<uint64_t *>(red + 4);    // [2][BQ], two blocks in turn
    int *rpos = reinterpret_cast<int *>(vmask2 + 2 * BQ), *rseq = rpos + BQ;
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, l16 = lane & 15, lg = lane >> 4;
    const int P = a.T * H, p0 = blockIdx.x * BQ;
    const int n_kv = *a.n_kv_dev;
    if (tid < 64) {
        int hi = 0;
        for (int i = tid; i < BQ; i += 64) {
            const bool live = p0 + i < P;
            const int t = live ? (p0 + i) / H : 0;
            rpos[i] = live ? a.tok_pos[t] : -1;
            rseq[i] = live ? (a.tok_seq[t] & 63) : -1;
            ms[i] = -INFINITY; ls[i] = 0.0f;
            if (live) { const int th = a.tok_hi ? (a.tok_hi[t] < n_kv ? a.tok_hi[t] : n_kv) : n_kv; hi = th > hi ? th : hi; }
        }
#pragma unroll
        for (int o = 32; o > 0; o >>= 1) hi = max(hi, __shfl_xor(hi, o, 64));
        if (tid == 0) red[0] = hi;
    }
    // the tile's queries (rows of P consecutive pairs: ld_qa = H kv_rank, ld_q = H (dim + rot)): the folded part as it is, the turning part turned; zeros behind
    // the row's length and for pairs past the end
    {
        const int K4 = KR >> 2, QD = a.dim + RT;
#pragma unroll 4
        for (int i = tid; i < BQ * K4; i += 64 * LT_NW) {
            const int r = i / K4, d = (i - r * K4) * 4;
            f32x4 v = {0.0f, 0.0f, 0.0f, 0.0f};
            if (p0 + r < P) v = *reinterpret_cast<const f32x4 *>(a.qa + (size_t)(p0 + r) * KR + d);
            *reinterpret_cast<f32x4 *>(Q + (size_t)r * LDQ + d) = f32x4{v.x * a.scale, v.y * a.scale, v.z * a.scale, v.w * a.scale};
        }
        const int half = a.rot_dims >> 1, rest = LQ - KR - a.rot_dims;
#pragma unroll 1
        for (int i = tid; i < BQ * half; i += 64 * LT_NW) {
            const int r = i / half, pr = i - r * half, p = p0 + r, iu = a.rot_halves ? pr : 2 * pr, iv = a.rot_halves ? pr + half : 2 * pr + 1;
            float x = 0.0f, y = 0.0f;
            if (p < P) {
                const float *qr = a.q + (size_t)p * QD + a.dim;
                const float u = qr[iu], w = qr[iv];
                float sn, c;
                sincosf((float)a.tok_pos[p / H] * a.rot_freq[pr], &sn, &c);
                sn *= a.rot_mscale * a.scale; c *= a.rot_mscale * a.scale;
                x = u * c - w * sn; y = w * c + u * sn;
            }
            Q[(size_t)r * LDQ + KR + iu] = x;
            Q[(size_t)r * LDQ + KR + iv] = y;
        }
#pragma unroll 1
        for (int i = tid; i < BQ * rest; i += 64 * LT_NW) {
            const int r = i / rest, e = a.rot_dims + i - r * rest;
            Q[(size_t)r * LDQ + KR + e] = p0 + r < P && e < RT ? a.q[(size_t)(p0 + r) * QD + a.dim + e] * a.scale : 0.0f;
        }
    }
    __syncthreads();
    int c_begin = 0, c_end = red[0];
    if (gridDim.y > 1) {
        const int per = ((c_end + BC - 1) / BC + (int)gridDim.y - 1) / (int)gridDim.y * BC;
        c_begin = (int)blockIdx.y * per;
        c_end = c_begin + per < c_end ? c_begin + per : c_end;
    }
    const int NJ = (KR + 63) >> 6;                              // tasks of the value pass: (J, row tile), J * R + tile
    f32x4 o[NT][4];
#pragma unroll
    for (int i = 0; i < NT; i++)
#pragma unroll
        for (int jj = 0; jj < 4; jj++) o[i][jj] = f32x4{0.0f, 0.0f, 0.0f, 0.0f};
    uint64_t *vmask = vmask2;
    for (int c0 = c_begin; c0 < c_end; c0 += BC) {
        vmask = vmask == vmask2 ? vmask2 + BQ : vmask2;          // (a slower wave may still be about to read the previous block's)
        int any = 0;
        {
            const int cc = c0 + lane;
            int cp = -1; uint64_t cs = 0;
            if (lane < BC && cc < c_end) { cp = a.cell_pos[cc]; cs = a.cell_seq[cc]; }
#pragma unroll
            for (int i = 0; i < 2 * R; i++) {
                const int r = wave + LT_NW * i, rp = rpos[r], rs = rseq[r];
                const bool v = cp >= 0 && rs >= 0 && cp <= rp && ((cs >> (rs & 63)) & 1) != 0 && !(a.window > 0 && rp - cp >= a.window);
                const uint64_t b = __ballot(v);
                if (lane == 0) vmask[r] = b;
                any |= b != 0;
            }
        }
        if (!__syncthreads_or(any)) continue;                   // (also: the previous block's weights have been used, the masks are in place)
        // ---- scores
        {
            constexpr int PIECES = lt_pieces(R, BC), PER = PIECES > LT_NW ? PIECES / LT_NW : 1;   // (PER row tiles of one cell piece per wave)
            const int piece = wave % (PIECES < LT_NW ? PIECES : LT_NW), ks = wave / (PIECES < LT_NW ? PIECES : LT_NW), s = piece % NS, rt0 = piece / NS;
            const int steps = LQ >> 4, per = (steps + KS - 1) / KS, u0 = ks * per, u1 = u0 + per < steps ? u0 + per : steps;
            const int c = c0 + 16 * s + l16;
            const float *kr = a.cache + (size_t)(c < c_end ? c : c_end - 1) * L + 4 * lg;
            const float *qr[PER];
            f32x4 acc[PER];
#pragma unroll
            for (int i = 0; i < PER; i++) { qr[i] = Q + (size_t)(16 * (rt0 + i * (LT_NW / NS)) + l16) * LDQ + 4 * lg; acc[i] = f32x4{0.0f, 0.0f, 0.0f, 0.0f}; }
#pragma unroll 4
            for (int u = u0; u < u1; u++) {
                const f32x4 k4 = 16 * u + 4 * lg < L ? *reinterpret_cast<const f32x4 *>(kr + 16 * u) : f32x4{0.0f, 0.0f, 0.0f, 0.0f};
#pragma unroll
                for (int i = 0; i < PER; i++) {
                    const f32x4 q4 = *reinterpret_cast<const f32x4 *>(qr[i] + 16 * u);
#pragma unroll
                    for (int e = 0; e < 4; e++) acc[i] = __builtin_amdgcn_mfma_f32_16x16x4f32(k4[e], q4[e], acc[i], 0, 0, 0);
                }
            }
#pragma unroll
            for (int i = 0; i < PER; i++) *reinterpret_cast<f32x4 *>(S + (size_t)(ks * BQ + 16 * (rt0 + i * (LT_NW / NS)) + l16) * LDS_S + 16 * s + 4 * lg) = acc[i];
        }
        __syncthreads();
        // ---- softmax: 16 lanes per pair
#pragma unroll 1
        for (int r = tid >> 4; r < BQ; r += 32) {
            const uint64_t seen = vmask[r];
            float x[NS];
            float bm = -INFINITY;
#pragma unroll
            for (int j = 0; j < NS; j++) {
                float v = S[(size_t)r * LDS_S + 16 * j + l16];
#pragma unroll
                for (int k = 1; k < KS; k++) v += S[(size_t)(k * BQ + r) * LDS_S + 16 * j + l16];
                x[j] = v;
                if ((seen >> (16 * j + l16)) & 1) bm = fmaxf(bm, v);
            }
            bm = fmaxf(bm, dpp_f<DPP_QP_1032>(bm));
            bm = fmaxf(bm, dpp_f<DPP_QP_2301>(bm));
            bm = fmaxf(bm, dpp_f<DPP_HALF_MIRROR>(bm));
            bm = fmaxf(bm, dpp_f<DPP_MIRROR>(bm));
            const float m0 = ms[r], mn = fmaxf(m0, bm), alpha = m0 == -INFINITY ? 0.0f : expf(m0 - mn);
            float ps = 0.0f;
#pragma unroll
            for (int j = 0; j < NS; j++) {
                const float p = (seen >> (16 * j + l16)) & 1 ? expf(x[j] - mn) : 0.0f;
                S[(size_t)r * LDS_S + 16 * j + l16] = p;
                ps += p;
            }
            ps = row_sum16(ps);
            if (l16 == 0) { ls[r] = ls[r] * alpha + ps; ms[r] = mn; al[r] = alpha; }
        }
        __syncthreads();
        // ---- values
#pragma unroll
        for (int i = 0; i < NT; i++) {
            const int task = wave + LT_NW * i;
            if (task >= NJ * R) continue;
            const int J = task / R, rt = task - J * R;
            const float alpha = al[16 * rt + l16];
#pragma unroll
            for (int jj = 0; jj < 4; jj++) { o[i][jj].x *= alpha; o[i][jj].y *= alpha; o[i][jj].z *= alpha; o[i][jj].w *= alpha; }
            const bool in = 64 * J + 4 * l16 < KR;
            const float *vb = a.cache + 64 * J + 4 * l16, *pb = S + (size_t)(16 * rt + l16) * LDS_S + 4 * lg;
            f32x4 v[4], vn[4];
            const auto fetch = [&](int s, f32x4 (&dst)[4]) {
#pragma unroll
                for (int e = 0; e < 4; e++) {
                    const int c = c0 + 16 * s + 4 * lg + e;      // (cells past the end repeat the last one with weight 0)
                    dst[e] = in ? *reinterpret_cast<const f32x4 *>(vb + (size_t)(c < c_end ? c : c_end - 1) * L) : f32x4{0.0f, 0.0f, 0.0f, 0.0f};
                }
            };
            fetch(0, v);
#pragma unroll 1
            for (int s = 0; s < NS; s++) {
                if (s + 1 < NS) fetch(s + 1, vn);
                const f32x4 p4 = *reinterpret_cast<const f32x4 *>(pb + 16 * s);
#pragma unroll
                for (int e = 0; e < 4; e++)
#pragma unroll
                    for (int jj = 0; jj < 4; jj++) o[i][jj] = __builtin_amdgcn_mfma_f32_16x16x4f32(v[e][jj], p4[e], o[i][jj], 0, 0, 0);
#pragma unroll
                for (int e = 0; e < 4; e++) v[e] = vn[e];
            }
        }
        // (no barrier: the next block's scores are written behind the barrier that ends its visibility test)
    }
    __syncthreads();
#pragma unroll
    for (int i = 0; i < NT; i++) {
        const int task = wave + LT_NW * i;
        if (task >= NJ * R) continue;
        const int J = task / R, rt = task - J * R, r = 16 * rt + l16, p = p0 + r;
        if (p >= P) continue;
        const int t = p / H, h = p - t * H;
        float *out, inv = 1.0f;
        if (gridDim.y > 1) {                                    // this run's record (sink and gate enter at the merge)
            out = a.part + ((size_t)p * gridDim.y + blockIdx.y) * (size_t)(KR + 2);
            if (J == 0 && lg == 0) *reinterpret_cast<float2 *>(out) = make_float2(ms[r], ls[r]);
            out += 2;
        } else {
            const float MM = a.sink ? fmaxf(ms[r], a.sink[h]) : ms[r];
            const float sc = ls[r] > 0.0f ? expf(ms[r] - MM) : 0.0f;
            const float den = ls[r] * sc + (a.sink ? expf(a.sink[h] - MM) : 0.0f);
            inv = latent_out_factor(a, t, h, den) * sc;
            out = a.out + (size_t)t * a.ld_out + (size_t)h * KR;
        }
#pragma unroll
        for (int rr = 0; rr < 4; rr++) {
            const int col = 64 * J + 16 * lg + 4 * rr;           // (kv_rank is a multiple of 4: four entries are inside or outside together)
            if (col >= KR) continue;
            *reinterpret_cast<float2 *>(out + col) = make_float2(o[i][0][rr] * inv, o[i][1][rr] * inv);
            *reinterpret_cast<float2 *>(out + col + 2) = make_float2(o[i][2][rr] * inv, o[i][3][rr] * inv);
        }
    }
}

template <int R, int BC, int NT>
static hipError_t launch_latent_tile(const LatentAttnArgs &a, hipStream_t st) {
    const int LQ = (a.kv_rank + a.rot + 15) & ~15;
    const size_t lds = lt_lds_floats(R, BC, LQ) * sizeof(float);
    if (lds > 60 * 1024) {
        const hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void *>(&latent_tile_kernel<R, BC, NT>), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds);
        if (e != hipSuccess) return e;
    }
    const long long P = (long long)a.T * a.H, tiles = (P + 16 * R - 1) / (16 * R);
    // enough runs of cells for two workgroups per CU; batches no more than there are blocks of cells (steps of few rows are launched for any number of cells)
    long long splits = (512 + tiles - 1) / tiles;
    if (BC == 64 && a.n_kv_hint > 0 && splits > (a.n_kv_hint + BC - 1) / BC) splits = (a.n_kv_hint + BC - 1) / BC;
    if (splits > (BC == 64 ? LATENT_TILE_RUNS : LATENT_STEP_RUNS)) splits = BC == 64 ? LATENT_TILE_RUNS : LATENT_STEP_RUNS;
    while (splits > 1 && (!a.part || (size_t)P * (size_t)splits * (a.kv_rank + 2) > a.part_floats)) splits--;
    hipLaunchKernelGGL((latent_tile_kernel<R, BC, NT>), dim3((unsigned)tiles, (unsigned)splits), dim3(64 * LT_NW), lds, st, a, LQ);
    return splits > 1 ? latent_attn_merge(a, (int)splits, st) : hipGetLastError();
}
template <int R, int BC>
static hipError_t launch_latent_tile_nt(const LatentAttnArgs &a, hipStream_t st) {
    const int tasks = (a.kv_rank + 63) / 64 * R;                 // (at most 17 R)
    if (tasks <= LT_NW) return launch_latent_tile<R, BC, 1>(a, st);
    if (tasks <= 2 * LT_NW) return launch_latent_tile<R, BC, 2>(a, st);
    if (tasks <= 4 * LT_NW) return launch_latent_tile<R, BC, 4>(a, st);
    return launch_latent_tile<R, BC, 9>(a, st);
}

}  // namespace

bool latent_attn_shape_ok(int kv_rank, int rot) { return kv_rank >= 1 && rot >= 0 && kv_rank + rot <= LA_MAX_L; }

hipError_t launch_latent_prep(const LatentPrepArgs &a, hipStream_t st) {
    if (a.T <= 0) return hipSuccess;
    if (a.rot_dims > a.rot || (a.rot_dims & 1)) return hipErrorInvalidValue;
    hipLaunchKernelGGL(latent_prep_kernel, dim3((unsigned)a.T), dim3(256), 0, st, a);
    return hipGetLastError();
}

hipError_t launch_latent_attn(const LatentAttnArgs &a, hipStream_t st) {
    if (a.T <= 0) return hipSuccess;
    if (!latent_attn_shape_ok(a.kv_rank, a.rot) || a.rot_dims > a.rot || (a.rot_dims & 1)) return hipErrorInvalidValue;
    const int L = a.kv_rank + a.rot;
    // rows that allow 16-byte loads take the matrix cores: batches in tiles of 32 (row, head) pairs (64 measured slower: fewer workgroups per CU) and blocks of 64 cells, steps of few pairs in
    // tiles of 16 or 32 pairs and blocks of 32 cells
    if ((L & 3) == 0 && (a.kv_rank & 3) == 0 && a.ld_qa == a.H * a.kv_rank && a.ld_q == a.H * (a.dim + a.rot) && (reinterpret_cast<uintptr_t>(a.qa) & 15) == 0 && (reinterpret_cast<uintptr_t>(a.cache) & 15) == 0) {
        const long long P = (long long)a.T * a.H;
        if (P <= 16) return launch_latent_tile_nt<1, 32>(a, st);
        if (P <= LATENT_STEP_MAX_PAIRS) return launch_latent_tile_nt<2, 32>(a, st);
        return launch_latent_tile_nt<2, 64>(a, st);
    }
    if (L <= 128) return launch_latent_attn_nj<2>(a, st);
    if (L <= 320) return launch_latent_attn_nj<5>(a, st);
    if (L <= 576) return launch_latent_attn_nj<9>(a, st);
    return launch_latent_attn_nj<17>(a, st);
}

}  // namespace mi355
