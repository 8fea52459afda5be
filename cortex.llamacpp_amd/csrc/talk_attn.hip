// talk_attn.hip — grouped-query attention whose heads mix their scores before the softmax ("talking heads"), on the f32 cache rows of gq_attn.hip.
//
//   score_h(i, j) = sum_g talk[h][g] (q_g,i . k_kv(g),j)          (the score's constant factors are part of the query)
//
// then everything as in gq_attn.hip: visibility from the cell table (same sequence, 0 <= pos_query - pos_cell < window or all earlier cells, the first
// keep_first positions of a window), softmax per head, an optional sink, the weighted sum of the head's own value head, an optional sigmoid gate per head.
// A head's softmax needs every head's score, so a workgroup works on ALL heads of its rows: the raw scores of a block of cells meet in LDS, are mixed there,
// and the mixed scores go on into the running softmax.  Keys and values are read once per group of heads that share them.  All f32.
//
// talk_row: steps of few rows - one workgroup per (row, run of cells).
// talk_tile: batches - one workgroup per (16 rows, run of cells, up to 8 * HPW heads to finish) on the f32 matrix cores (v_mfma_f32_16x16x4_f32: f32 operands,
// f32 accumulation, no reduced-precision mode).
// Both leave records [max | sum | weighted value] per (row, head, run) for gq_attn_merge where the cells are cut into several runs.
#include "kernels.h"

namespace mi355 {

namespace {

typedef float f32x4 __attribute__((ext_vector_type(4)));

// ---------------------------------------------------------------- a few rows
// A block of TKR_BC cells at a time, 8 waves.  Scores: 16 lanes per cell, 4 cells per wave, one key head after the other with the heads that read it (16-byte
// loads where the rows allow, the next key head in flight).  Mix: thread = (head, cell), a head's 32 cells are 32 neighbouring lanes, which also hold its softmax.
// Values: thread = (head, 4 columns) - or one column -, running sums in LDS.
constexpr int TKR_BC = 32, TKR_NT = 512;
constexpr int TKR_TALK_LDS = 64;                                // up to this many heads the mixing matrix is held in LDS too
constexpr size_t tkr_lds_floats(int H, int dim, int vdim) {
    return (size_t)H * dim + (size_t)H * (TKR_BC + 1) * 2 + (size_t)H * vdim + 3 * (size_t)H + 2 * TKR_BC + (H <= TKR_TALK_LDS ? (size_t)H * H : 0);
}
__device__ __forceinline__ float talk_half_max(float v) {       // over the 32 lanes of a half wave
    v = fmaxf(v, dpp_f<DPP_QP_1032>(v));
    v = fmaxf(v, dpp_f<DPP_QP_2301>(v));
    v = fmaxf(v, dpp_f<DPP_HALF_MIRROR>(v));
    v = fmaxf(v, dpp_f<DPP_MIRROR>(v));
    return fmaxf(v, __shfl_xor(v, 16, 64));
}

template <int NJ, bool VEC>
__global__ __launch_bounds__(TKR_NT) void talk_row_kernel(GqAttnArgs a) {
    extern __shared__ float lds[];
    const int H = a.H, G = a.G, D = a.dim, VD = a.vdim, HG = H / G;
    float *qv = lds, *acc = qv + (size_t)H * D, *raw = acc + (size_t)H * VD, *pw = raw + (size_t)H * (TKR_BC + 1), *ms = pw + (size_t)H * (TKR_BC + 1), *ls = ms + H, *al = ls + H;
    int *vis = reinterpret_cast<int *>(al + H);                  // [TKR_BC]
    float *tk = reinterpret_cast<float *>(vis + 2 * TKR_BC);     // [H][H]
    const float *talk = H <= TKR_TALK_LDS ? tk : a.talk;
    const int t = blockIdx.x, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, grp = lane >> 4, li = lane & 15;
    const size_t L = (size_t)G * (D + VD), voff = (size_t)G * D;
    const int tpos = a.tok_pos[t];
    const uint64_t sbit = 1ull << (a.tok_seq[t] & 63);
    int n_kv = *a.n_kv_dev;
    if (a.tok_hi) n_kv = a.tok_hi[t] < n_kv ? a.tok_hi[t] : n_kv;
    int c_lo = a.tok_lo ? a.tok_lo[t] : 0, c_hi = n_kv;
    if (c_lo > c_hi) c_lo = c_hi;
    if (gridDim.y > 1) {
        const int per = ((c_hi - c_lo + (int)gridDim.y - 1) / (int)gridDim.y + TKR_BC - 1) / TKR_BC * TKR_BC;
        c_lo += (int)blockIdx.y * per;
        c_hi = c_lo + per < c_hi ? c_lo + per : c_hi;
    }
    if (VEC) {
#pragma unroll 1
        for (int i = 4 * tid; i < H * D; i += 4 * TKR_NT) *reinterpret_cast<f32x4 *>(qv + i) = *reinterpret_cast<const f32x4 *>(a.q + (size_t)t * a.ld_q + i);
    } else {
#pragma unroll 1
        for (int i = tid; i < H * D; i += TKR_NT) qv[i] = a.q[(size_t)t * a.ld_q + i];
    }
#pragma unroll 1
    for (int i = tid; H <= TKR_TALK_LDS && i < H * H; i += TKR_NT) tk[i] = a.talk[i];
#pragma unroll 1
    for (int i = tid; i < H * VD; i += TKR_NT) acc[i] = 0.0f;
#pragma unroll 1
    for (int i = tid; i < H; i += TKR_NT) { ms[i] = -INFINITY; ls[i] = 0.0f; }
    const auto fetch = [&](int c, int kvh, float (&dst)[NJ][4]) {
        const float *kr = a.cache + (size_t)c * L + (size_t)kvh * D;
#pragma unroll
        for (int j = 0; j < NJ; j++) {
            const int e0 = 64 * j + 4 * li;
            if (VEC) {
                f32x4 v = {0.0f, 0.0f, 0.0f, 0.0f};
                if (c < c_hi && e0 < D) v = *reinterpret_cast<const f32x4 *>(kr + e0);
                dst[j][0] = v.x; dst[j][1] = v.y; dst[j][2] = v.z; dst[j][3] = v.w;
            } else {
#pragma unroll
                for (int e = 0; e < 4; e++) dst[j][e] = c < c_hi && e0 + e < D ? kr[e0 + e] : 0.0f;
            }
        }
    };
    for (int c0 = c_lo; c0 < c_hi; c0 += TKR_BC) {
        const int mine = wave * 4 + grp, c = c0 + mine;
        float ck[NJ][4], nk[NJ][4];
        fetch(c, 0, ck);                                         // (a cell of another sequence is read like any other; its score is dropped behind the mix)
        if (tid < TKR_BC) {
            const int cc = c0 + tid;
            const int cp = cc < c_hi ? a.cell_pos[cc] : -1;
            vis[tid] = cp >= 0 && cp <= tpos && (a.cell_seq[cc] & sbit) != 0 && !(a.window > 0 && tpos - cp >= a.window && cp >= a.keep_first);
        }
        __syncthreads();                                        // (queries are in place; the previous block's weights have been used)
        // ---- raw scores
        for (int kvh = 0; kvh < G; kvh++) {
            if (kvh + 1 < G) fetch(c, kvh + 1, nk);
#pragma unroll 2
            for (int g = kvh * HG; g < (kvh + 1) * HG; g++) {
                const float *q = qv + (size_t)g * D;
                float dot = 0.0f;
#pragma unroll
                for (int j = 0; j < NJ; j++) {
                    const int e0 = 64 * j + 4 * li;
                    if (VEC) {
                        if (e0 < D) {
                            const f32x4 q4 = *reinterpret_cast<const f32x4 *>(q + e0);
                            dot = fmaf(ck[j][0], q4.x, dot); dot = fmaf(ck[j][1], q4.y, dot); dot = fmaf(ck[j][2], q4.z, dot); dot = fmaf(ck[j][3], q4.w, dot);
                        }
                    } else {
#pragma unroll
                        for (int e = 0; e < 4; e++) if (e0 + e < D) dot = fmaf(ck[j][e], q[e0 + e], dot);
                    }
                }
                dot = row_sum16(dot);                            // over the cell's sixteen lanes
                if (li == 0) raw[g * (TKR_BC + 1) + mine] = dot;
            }
            if (kvh + 1 < G) {
#pragma unroll
                for (int j = 0; j < NJ; j++)
#pragma unroll
                    for (int e = 0; e < 4; e++) ck[j][e] = nk[j][e];
            }
        }
        __syncthreads();
        // ---- mixed scores and the running softmax: lane = cell, 32 lanes per head
#pragma unroll 1
        for (int idx = tid; idx < ((H * TKR_BC + 63) & ~63); idx += TKR_NT) {      // (whole waves: the shuffles below)
            const int h = idx / TKR_BC < H ? idx / TKR_BC : H - 1, cc = idx & (TKR_BC - 1);
            const float *tr = talk + (size_t)h * H;
            float s = 0.0f;
#pragma unroll 8
            for (int g = 0; g < H; g++) s = fmaf(tr[g], raw[g * (TKR_BC + 1) + cc], s);
            const bool seen = vis[cc] != 0;
            const float bm = talk_half_max(seen ? s : -INFINITY);
            const float m0 = ms[h], mn = fmaxf(m0, bm);
            const float p = seen ? expf(s - mn) : 0.0f;
            float ps = row_sum16(p);
            ps += __shfl_xor(ps, 16, 64);
            const float alpha = m0 == -INFINITY ? 0.0f : expf(m0 - mn);
            if (idx < H * TKR_BC) {
                pw[h * (TKR_BC + 1) + cc] = p;
                if (cc == 0) { ls[h] = ls[h] * alpha + ps; ms[h] = mn; al[h] = alpha; }   // (one wave holds the head's cells: every lane has read ms before)
            }
        }
        __syncthreads();
        // ---- weighted values
        const int nc = c_hi - c0 < TKR_BC ? c_hi - c0 : TKR_BC;
        if (VEC) {
            const int V4 = VD >> 2;
#pragma unroll 1
            for (int idx = tid; idx < H * V4; idx += TKR_NT) {
                const int h = idx / V4, col = (idx - h * V4) * 4;
                const float *vr = a.cache + (size_t)c0 * L + voff + (size_t)(h / HG) * VD + col, *p = pw + h * (TKR_BC + 1);
                f32x4 *o = reinterpret_cast<f32x4 *>(acc + (size_t)h * VD + col);
                const float alpha = al[h];
                f32x4 s = *o;
                s.x *= alpha; s.y *= alpha; s.z *= alpha; s.w *= alpha;
#pragma unroll 8
                for (int cc = 0; cc < nc; cc++) {
                    const f32x4 v = *reinterpret_cast<const f32x4 *>(vr + (size_t)cc * L);
                    const float w = p[cc];
                    s.x = fmaf(w, v.x, s.x); s.y = fmaf(w, v.y, s.y); s.z = fmaf(w, v.z, s.z); s.w = fmaf(w, v.w, s.w);
                }
                *o = s;
            }
        } else {
            for (int idx = tid; idx < H * VD; idx += TKR_NT) {
                const int h = idx / VD, col = idx - h * VD;
                const float *vr = a.cache + (size_t)c0 * L + voff + (size_t)(h / HG) * VD + col, *p = pw + h * (TKR_BC + 1);
                float s = acc[idx] * al[h];
#pragma unroll 8
                for (int cc = 0; cc < nc; cc++) s = fmaf(p[cc], vr[(size_t)cc * L], s);
                acc[idx] = s;
            }
        }
    }
    __syncthreads();
    if (gridDim.y > 1) {                                        // this run's records (sink and gate enter at the merge)
#pragma unroll 1
        for (int idx = tid; idx < H * (VD + 2); idx += TKR_NT) {
            const int h = idx / (VD + 2), i = idx - h * (VD + 2);
            a.part[(((size_t)t * H + h) * gridDim.y + blockIdx.y) * (size_t)(VD + 2) + i] = i == 0 ? ms[h] : i == 1 ? ls[h] : acc[(size_t)h * VD + i - 2];
        }
        return;
    }
#pragma unroll 1
    for (int idx = tid; idx < H * VD; idx += TKR_NT) {
        const int h = idx / VD;
        const float MM = a.sink ? fmaxf(ms[h], a.sink[h]) : ms[h];
        const float sc = ls[h] > 0.0f ? expf(ms[h] - MM) : 0.0f;
        const float den = ls[h] * sc + (a.sink ? expf(a.sink[h] - MM) : 0.0f);
        float inv = den > 0.0f ? sc / den : 0.0f;
        if (a.gate) inv *= 1.0f / (1.0f + expf(-a.gate[(size_t)t * a.ld_gate + h]));
        inv *= a.out_mult;
        a.out[(size_t)t * a.ld_out + idx] = acc[idx] * inv;
    }
}

// ---------------------------------------------------------------- batches
// 8 waves, BC cells per block.  v_mfma_f32_16x16x4_f32: lane l holds A[l & 15][l >> 4], B[l >> 4][l & 15], register r of the result is D[4 (l >> 4) + r][l & 15].
// The order of k inside a product is free as long as A and B agree, so a lane loads 4 consecutive floats (16 bytes) and feeds them to 4 products.
//   raw scores:  A = keys (i = cell), B = queries (j = row): a wave takes (head, half of the block's cells) tasks; result -> LDS, 4 cells of a row per write
//   mix:         A = talk (i = head, k = head), B = raw scores (k = head, j = (row, cell) pair): a wave owns 16 pairs at a time for ALL heads, so the mixed scores
//                take the raw ones' places without a barrier in between
//   softmax:     16 lanes per (head, row); weights back to LDS
//   values:      a wave owns heads (and, with few heads, a share of the value columns); A = values (i = column), B = weights (k = cell, j = row): the result's column is the lane's row, so the rescale needs no exchange; column i of
//                tile jj stands for value column 64 J + 4 i + jj, which makes every load 16 bytes and every lane's results 16 neighbouring columns
constexpr int TKT_NW = 8, TKT_BQ = 16;
constexpr int tkt_head_stride(int BC) { return TKT_BQ * (BC + 4) + 16; }
constexpr size_t tkt_lds_floats(int H, int BC) { return (size_t)(H + 1) * tkt_head_stride(BC) + 3 * (size_t)H * TKT_BQ + 2 * TKT_BQ + 4 + 4 * TKT_BQ; }   // (one more head: where the mix drops its padding)
constexpr size_t TKT_LDS_MAX = 156 * 1024;

// HPW: heads a wave finishes; NV = ceil(vdim / 64); the block's heads are [blockIdx.z * 8 * HPW, + 8 * HPW)
template <int BC, int HPW, int NV>
__global__ __launch_bounds__(64 * TKT_NW) void talk_tile_kernel(GqAttnArgs a, int wph) {
    constexpr int LDR = BC + 4, HS = tkt_head_stride(BC), NS = BC / 16, HT = BC == 64 ? 2 : 4;   // (at most 16 HT heads)
    extern __shared__ float lds[];
    const int H = a.H, G = a.G, D = a.dim, VD = a.vdim, HG = H / G;
    float *S = lds;                                             // [H + 1][16][LDR], head stride HS
    float *ms = S + (size_t)(H + 1) * HS, *ls = ms + H * TKT_BQ, *al = ls + H * TKT_BQ;      // [H][16]: running maximum and sum, this block's rescale
    int *rpos = reinterpret_cast<int *>(al + H * TKT_BQ), *rseq = rpos + TKT_BQ, *red = rseq + TKT_BQ;
    uint64_t *vmask2 = reinterpret_cast<uint64_t *>(red + 4);    // [2][16]: the cells of a block each row sees, two blocks in turn (an even number of floats in: 8-byte aligned)
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, l16 = lane & 15, lg = lane >> 4;
    const int row0 = blockIdx.x * TKT_BQ;
    const size_t L = (size_t)G * (D + VD), voff = (size_t)G * D;
    const int n_kv = *a.n_kv_dev;
#pragma unroll 1
    for (int i = tid; i < H * TKT_BQ; i += 64 * TKT_NW) { ms[i] = -INFINITY; ls[i] = 0.0f; }
    if (tid < 64) {
        int lo = 0x7fffffff, hi = 0;
        if (tid < TKT_BQ) {
            const int r = row0 + tid;
            const bool live = r < a.T;
            rpos[tid] = live ? a.tok_pos[r] : -1;
            rseq[tid] = live ? (a.tok_seq[r] & 63) : -1;
            if (live) {
                lo = a.tok_lo ? a.tok_lo[r] : 0;
                hi = a.tok_hi ? (a.tok_hi[r] < n_kv ? a.tok_hi[r] : n_kv) : n_kv;
            }
        }
#pragma unroll
        for (int o = 32; o > 0; o >>= 1) { lo = min(lo, __shfl_xor(lo, o, 64)); hi = max(hi, __shfl_xor(hi, o, 64)); }
        if (tid == 0) { red[0] = lo; red[1] = hi; }
    }
    __syncthreads();
    int c_begin = red[0] < red[1] ? red[0] : red[1], c_end = red[1];
    if (gridDim.y > 1) {
        const int per = ((c_end - c_begin + BC - 1) / BC + (int)gridDim.y - 1) / (int)gridDim.y * BC;
        c_begin += (int)blockIdx.y * per;
        c_end = c_begin + per < c_end ? c_begin + per : c_end;
    }
    // what this wave finishes: heads h0 + hh (hh < HPW), value columns of the 64-blocks J with J % wph == sub (wph waves share a head when there are few)
    const int sub = wave % wph, h0 = (int)blockIdx.z * TKT_NW * HPW + (wave / wph) * HPW;
    f32x4 o[HPW][NV][4];
#pragma unroll
    for (int hh = 0; hh < HPW; hh++)
#pragma unroll
        for (int J = 0; J < NV; J++)
#pragma unroll
            for (int jj = 0; jj < 4; jj++) o[hh][J][jj] = f32x4{0.0f, 0.0f, 0.0f, 0.0f};
    const float *qrow = a.q + (size_t)(row0 + l16 < a.T ? row0 + l16 : a.T - 1) * a.ld_q;    // (rows past the end repeat the last one and see nothing)
    uint64_t *vmask = vmask2;
    for (int c0 = c_begin; c0 < c_end; c0 += BC) {
        vmask = vmask == vmask2 ? vmask2 + TKT_BQ : vmask2;     // (a slower wave may still be about to read the previous block's)
        // ---- which cells each row sees: lane = cell, a wave tests rows wave and wave + 8
        int any = 0;
        {
            const int cc = c0 + lane;
            int cp = -1; uint64_t cs = 0;
            if (lane < BC && cc < c_end) { cp = a.cell_pos[cc]; cs = a.cell_seq[cc]; }
#pragma unroll
            for (int i = 0; i < 2; i++) {
                const int r = wave + 8 * i, rp = rpos[r];
                const bool v = cp >= 0 && rseq[r] >= 0 && cp <= rp && ((cs >> (rseq[r] & 63)) & 1) != 0 && !(a.window > 0 && rp - cp >= a.window && cp >= a.keep_first);
                const uint64_t b = __ballot(v);
                if (lane == 0) vmask[r] = b;
                any |= b != 0;
            }
        }
        if (!__syncthreads_or(any)) continue;                   // (also: the previous block's scores are no longer read, the masks are in place)
        // ---- raw scores
        for (int task = wave; task < 2 * H; task += TKT_NW) {
            const int g = task >> 1, s0 = (task & 1) * (NS / 2);
            const float *kb = a.cache + (size_t)(g / HG) * D, *qb = qrow + (size_t)g * D;
            const float *kr[NS / 2];
            f32x4 acc[NS / 2];
#pragma unroll
            for (int s = 0; s < NS / 2; s++) {
                const int c = c0 + 16 * (s0 + s) + l16;
                kr[s] = kb + (size_t)(c < c_end ? c : c_end - 1) * L;
                acc[s] = f32x4{0.0f, 0.0f, 0.0f, 0.0f};
            }
#pragma unroll 2
            for (int d0 = 0; d0 < D; d0 += 16) {                 // (dim is a multiple of 16)
                const int d = d0 + 4 * lg;
                const f32x4 q4 = *reinterpret_cast<const f32x4 *>(qb + d);
                f32x4 k4[NS / 2];
#pragma unroll
                for (int s = 0; s < NS / 2; s++) k4[s] = *reinterpret_cast<const f32x4 *>(kr[s] + d);
#pragma unroll
                for (int s = 0; s < NS / 2; s++)
#pragma unroll
                    for (int e = 0; e < 4; e++) acc[s] = __builtin_amdgcn_mfma_f32_16x16x4f32(k4[s][e], q4[e], acc[s], 0, 0, 0);
            }
#pragma unroll
            for (int s = 0; s < NS / 2; s++) *reinterpret_cast<f32x4 *>(S + (size_t)g * HS + l16 * LDR + 16 * (s0 + s) + 4 * lg) = acc[s];
        }
        __syncthreads();
        // ---- mix: four of the wave's column pieces side by side, so that the trip of a fragment of talk overlaps their products
#pragma unroll 1
        for (int ct0 = wave; ct0 < TKT_BQ * NS; ct0 += 4 * TKT_NW) {
            f32x4 mx[4][HT];
#pragma unroll
            for (int i = 0; i < 4; i++)
#pragma unroll
                for (int ht = 0; ht < HT; ht++) mx[i][ht] = f32x4{0.0f, 0.0f, 0.0f, 0.0f};
            const auto fragment = [&](int g0, float (&w)[HT]) {
#pragma unroll
                for (int ht = 0; ht < HT; ht++) w[ht] = g0 + lg < H && 16 * ht + l16 < H ? a.talk[(size_t)(16 * ht + l16) * H + g0 + lg] : 0.0f;
            };
            float w[HT], wn[HT];
            fragment(0, w);
            for (int g0 = 0; g0 < H; g0 += 4) {
                fragment(g0 + 4, wn);
                const bool in = g0 + lg < H;
#pragma unroll
                for (int i = 0; i < 4; i++) {
                    const int ct = ct0 + TKT_NW * i;
                    const float b = in ? S[(size_t)(g0 + lg) * HS + (ct / NS) * LDR + (ct % NS) * 16 + l16] : 0.0f;
#pragma unroll
                    for (int ht = 0; ht < HT; ht++) if (16 * ht < H) mx[i][ht] = __builtin_amdgcn_mfma_f32_16x16x4f32(w[ht], b, mx[i][ht], 0, 0, 0);
                }
#pragma unroll
                for (int ht = 0; ht < HT; ht++) w[ht] = wn[ht];
            }
#pragma unroll
            for (int i = 0; i < 4; i++) {
                const int ct = ct0 + TKT_NW * i;
                float *col = S + (ct / NS) * LDR + (ct % NS) * 16 + l16;
#pragma unroll
                for (int ht = 0; ht < HT; ht++) {
                    if (16 * ht >= H) continue;
#pragma unroll
                    for (int r = 0; r < 4; r++) {
                        const int h = 16 * ht + 4 * lg + r;
                        col[(size_t)(h < H ? h : H) * HS] = mx[i][ht][r];
                    }
                }
            }
        }
        __syncthreads();
        // ---- softmax: 16 lanes per (head, row)
#pragma unroll 1
        for (int hr = tid >> 4; hr < H * TKT_BQ; hr += 4 * TKT_NW) {
            const uint64_t seen = vmask[hr & (TKT_BQ - 1)] >> l16;
            float *row = S + (size_t)(hr >> 4) * HS + (hr & (TKT_BQ - 1)) * LDR + l16;
            float x[NS], bm = -INFINITY;
#pragma unroll
            for (int j = 0; j < NS; j++) {
                x[j] = (seen >> (16 * j)) & 1 ? row[16 * j] : -INFINITY;
                bm = fmaxf(bm, x[j]);
            }
            bm = fmaxf(bm, dpp_f<DPP_QP_1032>(bm));
            bm = fmaxf(bm, dpp_f<DPP_QP_2301>(bm));
            bm = fmaxf(bm, dpp_f<DPP_HALF_MIRROR>(bm));
            bm = fmaxf(bm, dpp_f<DPP_MIRROR>(bm));
            const float m0 = ms[hr], mn = fmaxf(m0, bm), mx = mn == -INFINITY ? 0.0f : mn;
            float ps = 0.0f;
#pragma unroll
            for (int j = 0; j < NS; j++) {
                const float p = expf(x[j] - mx);                 // (an unseen cell: e^-inf)
                row[16 * j] = p;
                ps += p;
            }
            ps = row_sum16(ps);
            const float alpha = expf(m0 - mx);                   // (nothing seen so far: e^-inf)
            if (l16 == 0) { ls[hr] = ls[hr] * alpha + ps; ms[hr] = mn; al[hr] = alpha; }
        }
        __syncthreads();
        // ---- values
#pragma unroll
        for (int hh = 0; hh < HPW; hh++) {
            const int h = h0 + hh;
            if (h >= H) continue;
            const float alpha = al[h * TKT_BQ + l16];
            const float *vb = a.cache + voff + (size_t)(h / HG) * VD + 4 * l16, *pb = S + (size_t)h * HS + l16 * LDR + 4 * lg;
#pragma unroll
            for (int J = 0; J < NV; J++) {
                if (J % wph != sub) continue;
#pragma unroll
                for (int jj = 0; jj < 4; jj++) { o[hh][J][jj].x *= alpha; o[hh][J][jj].y *= alpha; o[hh][J][jj].z *= alpha; o[hh][J][jj].w *= alpha; }
                const bool in = 64 * J + 4 * l16 < VD;
                f32x4 v[4], vn[4];
                const auto fetch = [&](int s, f32x4 (&dst)[4]) {
#pragma unroll
                    for (int e = 0; e < 4; e++) {
                        const int c = c0 + 16 * s + 4 * lg + e;  // (cells past the end repeat the last one with weight 0)
                        dst[e] = in ? *reinterpret_cast<const f32x4 *>(vb + (size_t)(c < c_end ? c : c_end - 1) * L + 64 * J) : f32x4{0.0f, 0.0f, 0.0f, 0.0f};
                    }
                };
                fetch(0, v);
#pragma unroll 1
                for (int s = 0; s < NS; s++) {
                    if (s + 1 < NS) fetch(s + 1, vn);
                    const f32x4 p = *reinterpret_cast<const f32x4 *>(pb + 16 * s);
#pragma unroll
                    for (int e = 0; e < 4; e++)
#pragma unroll
                        for (int jj = 0; jj < 4; jj++) o[hh][J][jj] = __builtin_amdgcn_mfma_f32_16x16x4f32(v[e][jj], p[e], o[hh][J][jj], 0, 0, 0);
#pragma unroll
                    for (int e = 0; e < 4; e++) v[e] = vn[e];
                }
            }
        }
        // (no barrier: the next block writes scores only behind the barrier that ends its visibility test)
    }
    // lane = (row l16, columns 64 J + 16 lg + 4 r + jj)
    __syncthreads();                                            // (a run without a visible cell has passed no barrier behind the start values of ms and ls)
    const int r = row0 + l16;
    if (r >= a.T) return;
#pragma unroll
    for (int hh = 0; hh < HPW; hh++) {
        const int h = h0 + hh;
        if (h >= H) continue;
        const float m = ms[h * TKT_BQ + l16], l = ls[h * TKT_BQ + l16];
        float *out, inv = 1.0f;
        if (gridDim.y > 1) {                                    // this run's record (sink and gate enter at the merge)
            out = a.part + (((size_t)r * H + h) * gridDim.y + blockIdx.y) * (size_t)(VD + 2);
            if (lg == 0 && sub == 0) *reinterpret_cast<float2 *>(out) = make_float2(m, l);
            out += 2;
        } else {
            const float MM = a.sink ? fmaxf(m, a.sink[h]) : m;
            const float sc = l > 0.0f ? expf(m - MM) : 0.0f;
            const float den = l * sc + (a.sink ? expf(a.sink[h] - MM) : 0.0f);
            inv = den > 0.0f ? sc / den : 0.0f;
            if (a.gate) inv *= 1.0f / (1.0f + expf(-a.gate[(size_t)r * a.ld_gate + h]));
            inv *= a.out_mult;
            out = a.out + (size_t)r * a.ld_out + (size_t)h * VD;
        }
#pragma unroll
        for (int J = 0; J < NV; J++) {
            if (J % wph != sub) continue;
#pragma unroll
            for (int rr = 0; rr < 4; rr++) {
                const int col = 64 * J + 16 * lg + 4 * rr;       // (vdim is a multiple of 4: four columns are inside or outside together)
                if (col >= VD) continue;
                *reinterpret_cast<float2 *>(out + col) = make_float2(o[hh][J][0][rr] * inv, o[hh][J][1][rr] * inv);
                *reinterpret_cast<float2 *>(out + col + 2) = make_float2(o[hh][J][2][rr] * inv, o[hh][J][3][rr] * inv);
            }
        }
    }
}

template <class K>
static hipError_t allow_lds(K *kernel, size_t bytes) {
    return bytes > 60 * 1024 ? hipFuncSetAttribute(reinterpret_cast<const void *>(kernel), hipFuncAttributeMaxDynamicSharedMemorySize, (int)bytes) : hipSuccess;
}

template <int NJ, bool VEC>
static hipError_t launch_talk_row(const GqAttnArgs &a, hipStream_t st) {
    const size_t lds = tkr_lds_floats(a.H, a.dim, a.vdim) * sizeof(float);
    hipError_t e = allow_lds(&talk_row_kernel<NJ, VEC>, lds);
    if (e != hipSuccess) return e;
    int splits = a.part ? TALK_ROW_RUNS / a.T : 1;
    splits = splits > TALK_ROW_SPLITS ? TALK_ROW_SPLITS : splits < 1 ? 1 : splits;
    while (splits > 1 && (size_t)a.T * a.H * splits * (a.vdim + 2) > a.part_floats) splits--;
    hipLaunchKernelGGL((talk_row_kernel<NJ, VEC>), dim3((unsigned)a.T, (unsigned)splits), dim3(TKR_NT), lds, st, a);
    return splits > 1 ? launch_gq_attn_merge(a, splits, st) : hipGetLastError();
}

template <int BC, int HPW, int NV>
static hipError_t launch_talk_tile(const GqAttnArgs &a, hipStream_t st) {
    const size_t lds = tkt_lds_floats(a.H, BC) * sizeof(float);
    hipError_t e = allow_lds(&talk_tile_kernel<BC, HPW, NV>, lds);
    if (e != hipSuccess) return e;
    // few heads and several 64-column blocks of values: the waves of a workgroup share heads instead of idling
    int wph = 1;
    while (HPW == 1 && wph * 2 <= NV && a.H * wph * 2 <= TKT_NW) wph *= 2;
    const long long tiles = (a.T + TKT_BQ - 1) / TKT_BQ, groups = (a.H + TKT_NW * HPW - 1) / (TKT_NW * HPW);
    long long splits = (512 + tiles * groups - 1) / (tiles * groups);
    const long long by_blocks = a.n_kv_hint > 0 ? (a.n_kv_hint + BC - 1) / BC : 1;
    if (splits > by_blocks) splits = by_blocks;
    if (splits > TALK_TILE_RUNS) splits = TALK_TILE_RUNS;
    while (splits > 1 && (!a.part || (size_t)a.T * a.H * splits * (a.vdim + 2) > a.part_floats)) splits--;
    if (splits < 1) splits = 1;
    hipLaunchKernelGGL((talk_tile_kernel<BC, HPW, NV>), dim3((unsigned)tiles, (unsigned)splits, (unsigned)groups), dim3(64 * TKT_NW), lds, st, a, wph);
    return splits > 1 ? launch_gq_attn_merge(a, (int)splits, st) : hipGetLastError();
}
template <int BC, int NV>
static hipError_t launch_talk_tile_h(const GqAttnArgs &a, hipStream_t st) {
    if (a.H <= 8) return launch_talk_tile<BC, 1, NV>(a, st);
    if (a.H <= 16 || NV > 2) return launch_talk_tile<BC, 2, NV>(a, st);
    return launch_talk_tile<BC, (NV > 2 ? 2 : 4), NV>(a, st);
}
template <int BC>
static hipError_t launch_talk_tile_bc(const GqAttnArgs &a, hipStream_t st) {
    if (a.vdim <= 64) return launch_talk_tile_h<BC, 1>(a, st);
    if (a.vdim <= 128) return launch_talk_tile_h<BC, 2>(a, st);
    return launch_talk_tile_h<BC, 4>(a, st);
}

}  // namespace

bool talk_attn_shape_ok(int H, int G, int dim, int vdim) { return gq_attn_shape_ok(H, G, dim, vdim) && tkr_lds_floats(H, dim, vdim) * sizeof(float) <= TKT_LDS_MAX; }

hipError_t launch_talk_attn(const GqAttnArgs &a, hipStream_t st) {
    if (a.T <= 0) return hipSuccess;
    if (!a.talk || a.maps > 1 || a.rel || a.v_cs || a.softcap > 0.0f || !talk_attn_shape_ok(a.H, a.G, a.dim, a.vdim)) return hipErrorInvalidValue;
    const auto al16 = [](const void *p) { return (reinterpret_cast<uintptr_t>(p) & 15) == 0; };
    const bool vec = (a.dim & 3) == 0 && (a.vdim & 3) == 0 && (a.ld_q & 3) == 0 && (a.ld_out & 3) == 0 && al16(a.q) && al16(a.out) && al16(a.cache);
    if (a.T >= 16 && vec && (a.dim & 15) == 0 && a.vdim <= 256 && a.H <= 64) {
        if (a.H <= 32 && tkt_lds_floats(a.H, 64) * sizeof(float) <= TKT_LDS_MAX) return launch_talk_tile_bc<64>(a, st);
        if (tkt_lds_floats(a.H, 32) * sizeof(float) <= TKT_LDS_MAX) return launch_talk_tile_bc<32>(a, st);
    }
    if (vec) {
        if (a.dim <= 64) return launch_talk_row<1, true>(a, st);
        if (a.dim <= 128) return launch_talk_row<2, true>(a, st);
        if (a.dim <= 256) return launch_talk_row<4, true>(a, st);
        return launch_talk_row<8, true>(a, st);
    }
    if (a.dim <= 64) return launch_talk_row<1, false>(a, st);
    if (a.dim <= 256) return launch_talk_row<4, false>(a, st);
    return launch_talk_row<8, false>(a, st);
}

}  // namespace mi355
