// mmb.hip — linear layers against BF16 weight rows ([out][in], K-contiguous) with f32 activations and f32 accumulation:
//
//   Y[z][t][n] = epi( sum_k X[z][t][k] * W[z][n][k] )
//
// z is an optional outer index with its own element strides on every operand: the heads of a per-head product (latent attention folds W_uk into the query
// and unfolds the attended latent through W_uv), the experts of a grouped batch (rows [offs[z], offs[z] + counts[z]) of X and Y belong to expert z), or
// the (token, rank) pairs of a few single tokens that picked their experts (sel[z] names the weight set, row z of Y, row z / sel_div of X).
//
// Three kernels behind one launch:
//   * mmb_vec   - up to a few dozen rows: one wave per output column walks K with 16-byte weight loads, the activations stay f32.  Weight-stream bound, the
//                 form of every single-token step in both precisions.
//   * mmb_mfma  - batches in bf16 mode: LDS-tiled, activations rounded to bf16 on the way in, v_mfma_f32_32x32x16_bf16, f32 accumulation.
//   * mmb_f32   - batches in f32 mode (and every shape the other two refuse): LDS-tiled, v_fma_f32 only - products of an f32 activation and a bf16 weight
//                 widened exactly, no reduced-precision matrix mode anywhere.
// Epilogues: store | relu(y)^2 | silu(W x) * (W2 x) | gelu_tanh(W x) * (W2 x) | g sigmoid(1.702 g) (u + 1) with g = W x capped from above and u = W2 x clamped
// to +- the same limit (the gated ones: two weight sets, one pass over the activations).  Around the epilogue, each optional: a factor per row on W x (and W2 x)
// - linear layers without a bias: the row of X itself times that number -, an f32 bias per output column in front of it, a residual row added behind it.  A
// grouped batch may read its rows of X, and write its rows of Y, through maps (no gather in front of the launch, no scatter behind it).
#include <type_traits>

#include "kernels.h"

namespace mi355 {

namespace {

typedef float f32x4 __attribute__((ext_vector_type(4)));
typedef float f32x16 __attribute__((ext_vector_type(16)));
typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));
typedef __bf16 bf16x4 __attribute__((ext_vector_type(4)));
typedef unsigned short u16x8 __attribute__((ext_vector_type(8)));
typedef unsigned short u16x4 __attribute__((ext_vector_type(4)));

__device__ __forceinline__ float bf2f(unsigned short h) { return __uint_as_float((unsigned)h << 16); }
__device__ __forceinline__ float epi_apply(int epi, float a, float b, float lim = 0.0f) {
    if (epi == MMB_CLAMP_SWIGLU) {
        const float g = fminf(a, lim), u = fminf(fmaxf(b, -lim), lim);
        return g / (1.0f + expf(-1.702f * g)) * (u + 1.0f);
    }
    if (epi == MMB_RELU2) { const float r = a > 0.0f ? a : 0.0f; return r * r; }
    if (epi == MMB_SILU_MUL) return a / (1.0f + expf(-a)) * b;
    if (epi == MMB_GELU_MUL) return 0.5f * a * (1.0f + tanhf(0.7978845608028654f * (a + 0.044715f * a * a * a))) * b;   // the tanh form of gelu; sqrt(2 / pi)
    return a;
}

// the epilogue as a template argument: a workgroup's finished tile runs through its code once, so what is not asked for should not lie in between (EPI_ANY: a.epi)
constexpr int EPI_ANY = -1;
template <int EPI> __device__ __forceinline__ float epi_fixed(const MMBArgs &a, float s1, float s2) { return epi_apply(EPI == EPI_ANY ? a.epi : EPI, s1, s2, a.epi_limit); }

// where the rows of outer index z live: first row and row count of X / Y, the weight set
struct ZView { const float *x; const unsigned short *w, *w2; float *y; const float *resid; int rows, x0, y0; };   // x, y, resid: bases; row t of z: x0 + t, y0 + t
__device__ __forceinline__ ZView z_view(const MMBArgs &a, int z) {
    ZView v;
    int wz = z;
    v.x0 = v.y0 = 0;
    v.rows = a.T;
    if (a.sel) { wz = a.sel[z]; v.x0 = z / a.sel_div; v.y0 = z; v.rows = 1; }
    else if (a.meta) { v.rows = a.meta[z]; v.x0 = v.y0 = a.meta[a.nz + z]; }
    v.x = a.x + (size_t)(a.sel || a.meta ? 0 : z) * a.x_zs;
    v.y = a.y + (size_t)(a.sel || a.meta ? 0 : z) * a.y_zs;
    v.resid = a.resid ? a.resid + (size_t)(a.sel || a.meta ? 0 : z) * a.y_zs : nullptr;
    v.w = a.w + (size_t)wz * a.w_zs;
    v.w2 = a.w2 ? a.w2 + (size_t)wz * a.w_zs : nullptr;
    return v;
}

__device__ __forceinline__ const float *x_row(const MMBArgs &a, const ZView &v, int t) { return v.x + (size_t)(a.x_map ? a.x_map[v.x0 + t] : v.x0 + t) * a.ldx; }
__device__ __forceinline__ size_t y_row(const MMBArgs &a, const ZView &v, int t) { return (size_t)(a.y_map ? a.y_map[v.y0 + t] : v.y0 + t) * a.ldy; }
// output (t, n) from its finished sums; yr = y_row(t), rs = the row's factor, res = the residual's entry (0: none)
template <int EPI>
__device__ __forceinline__ void y_store(const MMBArgs &a, const ZView &v, size_t yr, int n, float s1, float s2, float rs, float res) {
    s1 *= rs; s2 *= rs;
    v.y[yr + n] = epi_fixed<EPI>(a, a.bias ? s1 + a.bias[n] : s1, s2) * a.out_scale + res;
}

// ---- the layer norm of a row inside a product (LN): the walk over k sums (x - c) w_k g_k, (x - c) and (x - c)^2 around a value c near the row's mean - the mean of its
// first entries, so that nothing is lost in the difference of large sums -, and what is left follows from the column's own sums with the norm's weight and bias
template <bool VEC>
__device__ __forceinline__ float row_middle(const float *x, int K, int lane) {
    float s = 0.0f;
    if (VEC) {
        if (lane * 8 < K) {
            const f32x4 u = *reinterpret_cast<const f32x4 *>(x + lane * 8), w = *reinterpret_cast<const f32x4 *>(x + lane * 8 + 4);
            s = ((u.x + u.y) + (u.z + u.w)) + ((w.x + w.y) + (w.z + w.w));
        }
    } else s = lane < K ? x[lane] : 0.0f;
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) s += __shfl_xor(s, o, 64);
    const int n = VEC ? 512 : 64;
    return s / (float)(K < n ? K : n);
}
__device__ __forceinline__ float row_offset(float sx, int K) {  // mean - c
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) sx += __shfl_xor(sx, o, 64);
    return sx / (float)K;
}
__device__ __forceinline__ float ln_close(float s, float off, float inv, const float *ln, int n, int N) { return fmaf(s - off * ln[n], inv, ln[N + n]); }

// ---------------------------------------------------------------- few rows: one wave per output column
// Few rows against MANY output columns (single-token steps: the head, the feed-forward): a wave owns NR adjacent weight rows and keeps the activations of a
// 512-wide piece of k in registers for all of them - the activation and norm-weight loads, which every wave repeats out of the caches, are paid once per NR
// weight rows instead of once per row.  Up to TBR rows of X; 16-byte aligned operands; same arithmetic per output as mmb_vec_kernel.
template <int NR, int TBR, int EPI, bool LN>
__global__ __launch_bounds__(256) void mmb_vec_rows_kernel(MMBArgs a) {
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    const int n0 = (blockIdx.x * 4 + wave) * NR;
    const ZView v = z_view(a, blockIdx.y);
    if (n0 >= a.N) return;
    const bool pn = a.pn_w != nullptr, gated = v.w2 != nullptr;
    const unsigned short *wr[NR], *wr2[NR];
#pragma unroll
    for (int r = 0; r < NR; r++) {
        const int n = n0 + r < a.N ? n0 + r : a.N - 1;          // rows past the end read the last row; their results are never stored
        wr[r] = v.w + (size_t)n * a.ldw;
        wr2[r] = gated ? v.w2 + (size_t)n * a.ldw : wr[r];
    }
    float acc[NR][TBR], acc2[NR][TBR], ss[TBR], sx[LN ? TBR : 1], mid[LN ? TBR : 1];
#pragma unroll
    for (int i = 0; i < TBR; i++) {
        ss[i] = 0.0f;
        if (LN) sx[i] = 0.0f;
#pragma unroll
        for (int r = 0; r < NR; r++) { acc[r][i] = 0.0f; acc2[r][i] = 0.0f; }
    }
    const int nt = v.rows < TBR ? v.rows : TBR;
    float res[NR][TBR], rsc[TBR];                               // (requested in front of the walk over k: nothing waits for them behind it)
#pragma unroll
    for (int i = 0; i < TBR; i++) {
        rsc[i] = a.row_scale && i < nt ? a.row_scale[v.y0 + i] : 1.0f;
#pragma unroll
        for (int r = 0; r < NR; r++) res[r][i] = v.resid && i < nt && n0 + r < a.N ? v.resid[y_row(a, v, i) + n0 + r] : 0.0f;
    }
    u16x8 w8n[NR], w28n[NR];                                    // (LN: a piece's weights are on their way while the rows' middle values, or the piece before, are worked on)
#pragma unroll
    for (int r = 0; r < NR; r++) w8n[r] = w28n[r] = u16x8{0, 0, 0, 0, 0, 0, 0, 0};
    const auto ahead = [&](int k) {
        if (k >= a.K) return;
#pragma unroll
        for (int r = 0; r < NR; r++) {
            w8n[r] = *reinterpret_cast<const u16x8 *>(wr[r] + k);
            if (gated) w28n[r] = *reinterpret_cast<const u16x8 *>(wr2[r] + k);
        }
    };
    if (LN) {
        ahead(lane * 8);
#pragma unroll
        for (int i = 0; i < TBR; i++) mid[i] = i < nt ? row_middle<true>(x_row(a, v, i), a.K, lane) : 0.0f;
    }
    for (int k = lane * 8; k < a.K; k += 512) {
        if (!LN) ahead(k);
        u16x8 w8[NR], w28[NR];
#pragma unroll
        for (int r = 0; r < NR; r++) { w8[r] = w8n[r]; w28[r] = w28n[r]; }
        if (LN) ahead(k + 512);
        float pw[8];
        if (pn) {
            const f32x4 g0 = *reinterpret_cast<const f32x4 *>(a.pn_w + k), g1 = *reinterpret_cast<const f32x4 *>(a.pn_w + k + 4);
            pw[0] = a.pn_off + g0.x; pw[1] = a.pn_off + g0.y; pw[2] = a.pn_off + g0.z; pw[3] = a.pn_off + g0.w;
            pw[4] = a.pn_off + g1.x; pw[5] = a.pn_off + g1.y; pw[6] = a.pn_off + g1.z; pw[7] = a.pn_off + g1.w;
        }
#pragma unroll
        for (int i = 0; i < TBR; i++) {
            if (i >= nt) break;
            const float *xr = x_row(a, v, i) + k;
            const f32x4 x0 = *reinterpret_cast<const f32x4 *>(xr), x1 = *reinterpret_cast<const f32x4 *>(xr + 4);
            float xs[8] = {x0.x, x0.y, x0.z, x0.w, x1.x, x1.y, x1.z, x1.w};
            if (LN) {
#pragma unroll
                for (int e = 0; e < 8; e++) { xs[e] -= mid[i]; sx[i] += xs[e]; }
            }
            if (pn) {
#pragma unroll
                for (int e = 0; e < 8; e++) { ss[i] = fmaf(xs[e], xs[e], ss[i]); xs[e] = xs[e] * pw[e]; }
            }
#pragma unroll
            for (int r = 0; r < NR; r++)
#pragma unroll
                for (int e = 0; e < 8; e++) {
                    acc[r][i] = fmaf(xs[e], bf2f(w8[r][e]), acc[r][i]);
                    if (gated) acc2[r][i] = fmaf(xs[e], bf2f(w28[r][e]), acc2[r][i]);
                }
        }
    }
#pragma unroll
    for (int i = 0; i < TBR; i++) {
        if (i >= nt) break;
        float q = ss[i];
#pragma unroll
        for (int o = 32; o > 0; o >>= 1) q += __shfl_xor(q, o, 64);
        const float off = LN ? row_offset(sx[i], a.K) : 0.0f;
        const float inv = pn ? 1.0f / sqrtf(q / (float)a.K - off * off + a.pn_eps) : 1.0f;
#pragma unroll
        for (int r = 0; r < NR; r++) {
            float s1 = acc[r][i], s2 = acc2[r][i];
#pragma unroll
            for (int o = 32; o > 0; o >>= 1) { s1 += __shfl_xor(s1, o, 64); s2 += __shfl_xor(s2, o, 64); }
            if (LN) { const int n = n0 + r < a.N ? n0 + r : a.N - 1; s1 = ln_close(s1, off, inv, a.ln, n, a.N); if (gated) s2 = ln_close(s2, off, inv, a.ln2, n, a.N); }
            else if (pn) { s1 *= inv; s2 *= inv; }
            if (lane == 0 && n0 + r < a.N) y_store<EPI>(a, v, y_row(a, v, i), n0 + r, s1, s2, rsc[i], res[r][i]);
        }
    }
}

// With the norm prologue the row's sum of squares is gathered in the same pass as the products: y = inv_rms(x) * sum_k w_k (x_k (off + g_k)) - one trip
// through memory per wave, the scale applied to the finished sum.
// TB: rows per pass - 1 for single rows (a short program: a step runs it once per launch, its first fetch is part of the time), else 8
template <bool VEC, int TB, int EPI, bool LN>
__global__ __launch_bounds__(256) void mmb_vec_kernel(MMBArgs a) {
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    const int n = blockIdx.x * 4 + wave;
    const ZView v = z_view(a, blockIdx.y);
    if (n >= a.N) return;
    const unsigned short *wr = v.w + (size_t)n * a.ldw, *wr2 = v.w2 ? v.w2 + (size_t)n * a.ldw : nullptr;
    const bool pn = a.pn_w != nullptr;
    for (int t0 = 0; t0 < v.rows; t0 += TB) {
        float acc[TB], acc2[TB], ss[TB], sx[LN ? TB : 1], mid[LN ? TB : 1];
#pragma unroll
        for (int i = 0; i < TB; i++) { acc[i] = 0.0f; acc2[i] = 0.0f; ss[i] = 0.0f; if (LN) sx[i] = 0.0f; }
        const int nt = v.rows - t0 < TB ? v.rows - t0 : TB;
        float res[TB], rsc[TB];
#pragma unroll
        for (int i = 0; i < TB; i++) {
            rsc[i] = a.row_scale && i < nt ? a.row_scale[v.y0 + t0 + i] : 1.0f;
            res[i] = v.resid && i < nt ? v.resid[y_row(a, v, t0 + i) + n] : 0.0f;
        }
        u16x8 w8n = {0, 0, 0, 0, 0, 0, 0, 0}, w28n = w8n;           // (LN: a piece's weights are on their way while the row's middle value, or the piece before, is worked on)
        const auto ahead = [&](int k) {
            if (k >= a.K) return;
            w8n = *reinterpret_cast<const u16x8 *>(wr + k);
            if (wr2) w28n = *reinterpret_cast<const u16x8 *>(wr2 + k);
        };
        if (LN) {
            if (VEC) ahead(lane * 8);
#pragma unroll
            for (int i = 0; i < TB; i++) mid[i] = i < nt ? row_middle<VEC>(x_row(a, v, t0 + i), a.K, lane) : 0.0f;
        }
        if (VEC) {
            for (int k = lane * 8; k < a.K; k += 512) {
                if (!LN) ahead(k);
                const u16x8 w8 = w8n, w28 = w28n;
                if (LN) ahead(k + 512);
                float pw[8];
                if (pn) {
                    const f32x4 g0 = *reinterpret_cast<const f32x4 *>(a.pn_w + k), g1 = *reinterpret_cast<const f32x4 *>(a.pn_w + k + 4);
                    pw[0] = a.pn_off + g0.x; pw[1] = a.pn_off + g0.y; pw[2] = a.pn_off + g0.z; pw[3] = a.pn_off + g0.w;
                    pw[4] = a.pn_off + g1.x; pw[5] = a.pn_off + g1.y; pw[6] = a.pn_off + g1.z; pw[7] = a.pn_off + g1.w;
                }
#pragma unroll
                for (int i = 0; i < TB; i++) {
                    if (i >= nt) break;
                    const float *xr = x_row(a, v, t0 + i) + k;
                    const f32x4 x0 = *reinterpret_cast<const f32x4 *>(xr), x1 = *reinterpret_cast<const f32x4 *>(xr + 4);
                    float xs[8] = {x0.x, x0.y, x0.z, x0.w, x1.x, x1.y, x1.z, x1.w};
                    if (LN) {
#pragma unroll
                        for (int e = 0; e < 8; e++) { xs[e] -= mid[i]; sx[i] += xs[e]; }
                    }
                    if (pn) {
#pragma unroll
                        for (int e = 0; e < 8; e++) { ss[i] = fmaf(xs[e], xs[e], ss[i]); xs[e] = xs[e] * pw[e]; }
                    }
#pragma unroll
                    for (int e = 0; e < 8; e++) {
                        acc[i] = fmaf(xs[e], bf2f(w8[e]), acc[i]);
                        if (wr2) acc2[i] = fmaf(xs[e], bf2f(w28[e]), acc2[i]);
                    }
                }
            }
        } else {
            for (int k = lane; k < a.K; k += 64) {
                const float w = bf2f(wr[k]), w2 = wr2 ? bf2f(wr2[k]) : 0.0f, pw = pn ? a.pn_off + a.pn_w[k] : 1.0f;
#pragma unroll
                for (int i = 0; i < TB; i++) {
                    if (i >= nt) break;
                    float x = x_row(a, v, t0 + i)[k];
                    if (LN) { x -= mid[i]; sx[i] += x; }
                    if (pn) { ss[i] = fmaf(x, x, ss[i]); x = x * pw; }
                    acc[i] = fmaf(x, w, acc[i]);
                    acc2[i] = fmaf(x, w2, acc2[i]);
                }
            }
        }
#pragma unroll
        for (int i = 0; i < TB; i++) {
            if (i >= nt) break;
            float s = acc[i], s2 = acc2[i], q = ss[i];
#pragma unroll
            for (int o = 32; o > 0; o >>= 1) { s += __shfl_xor(s, o, 64); s2 += __shfl_xor(s2, o, 64); q += __shfl_xor(q, o, 64); }
            if (LN) {
                const float off = row_offset(sx[i], a.K), inv = 1.0f / sqrtf(q / (float)a.K - off * off + a.pn_eps);
                s = ln_close(s, off, inv, a.ln, n, a.N);
                if (wr2) s2 = ln_close(s2, off, inv, a.ln2, n, a.N);
            } else if (pn) { const float inv = 1.0f / sqrtf(q / (float)a.K + a.pn_eps); s *= inv; s2 *= inv; }
            if (lane == 0) y_store<EPI>(a, v, y_row(a, v, t0 + i), n, s, s2, rsc[i], res[i]);
        }
    }
}

// ---------------------------------------------------------------- batches, f32: 64 x 64 outputs per workgroup, 16 of k per stage, 4 x 4 per thread
template <bool GATED>
__global__ __launch_bounds__(256) void mmb_f32_kernel(MMBArgs a) {
    constexpr int BM = 64, BN = 64, BK = 16, LD = 68;
    __shared__ float sX[BK][LD], sW[BK][LD], sW2[GATED ? BK : 1][LD];
    const ZView v = z_view(a, blockIdx.z);
    const int t0 = blockIdx.y * BM, n0 = blockIdx.x * BN;
    if (t0 >= v.rows) return;                                   // (uniform: before any barrier)
    const int tid = threadIdx.x, tx = tid & 15, ty = tid >> 4;
    const int lr = tid >> 2, lk = (tid & 3) * 4;                 // loader: row lr of both tiles, 4 consecutive k
    float acc[4][4], acc2[4][4];
#pragma unroll
    for (int i = 0; i < 4; i++)
#pragma unroll
        for (int j = 0; j < 4; j++) { acc[i][j] = 0.0f; acc2[i][j] = 0.0f; }
    const bool xrow = t0 + lr < v.rows, wrow = n0 + lr < a.N;
    const float *xr = x_row(a, v, xrow ? t0 + lr : t0);
    const unsigned short *wr = v.w + (size_t)(n0 + lr) * a.ldw;
    const unsigned short *wr2 = GATED ? v.w2 + (size_t)(n0 + lr) * a.ldw : nullptr;
    for (int k0 = 0; k0 < a.K; k0 += BK) {
#pragma unroll
        for (int e = 0; e < 4; e++) {
            const int k = k0 + lk + e;
            const bool in = k < a.K;
            sX[lk + e][lr] = xrow && in ? xr[k] : 0.0f;
            sW[lk + e][lr] = wrow && in ? bf2f(wr[k]) : 0.0f;
            if (GATED) sW2[lk + e][lr] = wrow && in ? bf2f(wr2[k]) : 0.0f;
        }
        __syncthreads();
#pragma unroll
        for (int k = 0; k < BK; k++) {
            const f32x4 xv = *reinterpret_cast<const f32x4 *>(&sX[k][ty * 4]);
            const f32x4 wv = *reinterpret_cast<const f32x4 *>(&sW[k][tx * 4]);
            const float xs[4] = {xv.x, xv.y, xv.z, xv.w}, ws[4] = {wv.x, wv.y, wv.z, wv.w};
#pragma unroll
            for (int i = 0; i < 4; i++)
#pragma unroll
                for (int j = 0; j < 4; j++) acc[i][j] = fmaf(xs[i], ws[j], acc[i][j]);
            if (GATED) {
                const f32x4 w2v = *reinterpret_cast<const f32x4 *>(&sW2[k][tx * 4]);
                const float w2s[4] = {w2v.x, w2v.y, w2v.z, w2v.w};
#pragma unroll
                for (int i = 0; i < 4; i++)
#pragma unroll
                    for (int j = 0; j < 4; j++) acc2[i][j] = fmaf(xs[i], w2s[j], acc2[i][j]);
            }
        }
        __syncthreads();
    }
#pragma unroll
    for (int i = 0; i < 4; i++) {
        const int t = t0 + ty * 4 + i;
        if (t >= v.rows) continue;
        const size_t yr = y_row(a, v, t);
        const float rs = a.row_scale ? a.row_scale[v.y0 + t] : 1.0f;
#pragma unroll
        for (int j = 0; j < 4; j++) {
            const int n = n0 + tx * 4 + j;
            if (n < a.N) y_store<EPI_ANY>(a, v, yr, n, acc[i][j], acc2[i][j], rs, v.resid ? v.resid[yr + n] : 0.0f);
        }
    }
}

// ---------------------------------------------------------------- batches, bf16 on the matrix cores
// 64 RN weight rows x 64 RT rows of X per workgroup, 64 of k per stage: both operands through LDS (two buffers, one barrier per stage; rows padded to an odd number
// of 16-byte pieces), X rounded to bf16 once on its way there, the stages after next already on their way from memory in registers.  A wave owns 32 RN x 32 RT
// outputs (v_mfma_f32_32x32x16_bf16).  The workgroups that read the same weight rows sit on the same XCD, side by side: its L2 fetches them once.
constexpr int MMT_K = 64, MMT_LD = MMT_K + 8;                   // bf16 per LDS row
template <int RN, int RT, int EPI>
__global__ __launch_bounds__(256) void mmb_mfma_kernel(MMBArgs a, int n_tiles, int t_tiles) {
    constexpr bool GATED = EPI >= MMB_SILU_MUL;
    constexpr int TN = 64 * RN, TT = 64 * RT, NW = 2 * RN, NX = 4 * RT;   // 16-byte loads per thread and stage
    constexpr int SETS = RN * RT == 1 ? 4 : 2;                  // stages on their way from memory
    __shared__ __attribute__((aligned(16))) unsigned short sW[2][TN][MMT_LD], sW2[GATED ? 2 : 1][GATED ? TN : 1][MMT_LD], sX[2][TT][MMT_LD];
    const ZView v = z_view(a, blockIdx.z);
    // block -> tile: consecutive blocks go to the XCDs in turn; the t tiles of one n tile take consecutive turns of ONE of them
    const int xcd = blockIdx.x & 7, turn = blockIdx.x >> 3, nt = xcd + 8 * (turn / t_tiles), n0 = nt * TN, t0 = (turn % t_tiles) * TT;
    if (nt >= n_tiles || t0 >= v.rows) return;                  // (uniform: before any barrier)
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, m = lane & 31, kg = lane >> 5;
    const int r4 = tid >> 2, q4 = tid & 3;
    const unsigned short *wr[RN], *wr2[RN];
    const float *xr[RT];
#pragma unroll
    for (int i = 0; i < RN; i++) {
        const int n = n0 + 64 * i + r4 < a.N ? n0 + 64 * i + r4 : a.N - 1;          // rows past the end read the last row; their results are never stored
        wr[i] = v.w + (size_t)n * a.ldw + 8 * q4;
        wr2[i] = GATED ? v.w2 + (size_t)n * a.ldw + 8 * q4 : nullptr;
    }
#pragma unroll
    for (int i = 0; i < RT; i++) { const int t = t0 + 64 * i + r4; xr[i] = x_row(a, v, t < v.rows ? t : v.rows - 1) + 4 * q4; }
    f32x16 acc[RN][RT], acc2[GATED ? RN : 1][GATED ? RT : 1];
#pragma unroll
    for (int i = 0; i < RN; i++)
#pragma unroll
        for (int j = 0; j < RT; j++)
#pragma unroll
            for (int r = 0; r < 16; r++) { acc[i][j][r] = 0.0f; if (GATED) acc2[i][j][r] = 0.0f; }
    u16x8 lw[SETS][NW], lw2[SETS][GATED ? NW : 1];
    f32x4 lx[SETS][NX];
    const auto request = [&](auto set, int k0) {                // (K is a multiple of 16: a 16-byte piece is inside a row or behind its end)
        constexpr int b = decltype(set)::value;
#pragma unroll
        for (int i = 0; i < NW; i++) {
            const int k = k0 + 32 * (i & 1);
            const bool in = k + 8 * q4 < a.K;
            lw[b][i] = in ? *reinterpret_cast<const u16x8 *>(wr[i >> 1] + k) : u16x8{0, 0, 0, 0, 0, 0, 0, 0};
            if (GATED) lw2[b][i] = in ? *reinterpret_cast<const u16x8 *>(wr2[i >> 1] + k) : u16x8{0, 0, 0, 0, 0, 0, 0, 0};
        }
#pragma unroll
        for (int i = 0; i < NX; i++) {
            const int k = k0 + 16 * (i & 3);
            lx[b][i] = k < a.K ? *reinterpret_cast<const f32x4 *>(xr[i >> 2] + k) : f32x4{0.0f, 0.0f, 0.0f, 0.0f};
        }
    };
    const auto stage = [&](auto set) {
        constexpr int w = decltype(set)::value, b = w & 1;
#pragma unroll
        for (int i = 0; i < NW; i++) {
            *reinterpret_cast<u16x8 *>(&sW[b][64 * (i >> 1) + r4][32 * (i & 1) + 8 * q4]) = lw[w][i];
            if (GATED) *reinterpret_cast<u16x8 *>(&sW2[b][64 * (i >> 1) + r4][32 * (i & 1) + 8 * q4]) = lw2[w][i];
        }
#pragma unroll
        for (int i = 0; i < NX; i++) {
            const f32x4 x = lx[w][i];
            *reinterpret_cast<bf16x4 *>(&sX[b][64 * (i >> 2) + r4][16 * (i & 3) + 4 * q4]) = bf16x4{(__bf16)x.x, (__bf16)x.y, (__bf16)x.z, (__bf16)x.w};   // (round to nearest even)
        }
    };
    const auto multiply = [&](auto set) {
        constexpr int b = decltype(set)::value & 1;
#pragma unroll
        for (int u = 0; u < MMT_K / 16; u++) {
            bf16x8 wa[RN], wb[RN], xb[RT];
#pragma unroll
            for (int i = 0; i < RN; i++) {
                const int n = (wave & 1) * 32 * RN + 32 * i + m;
                wa[i] = *reinterpret_cast<const bf16x8 *>(&sW[b][n][16 * u + 8 * kg]);
                if (GATED) wb[i] = *reinterpret_cast<const bf16x8 *>(&sW2[b][n][16 * u + 8 * kg]);
            }
#pragma unroll
            for (int j = 0; j < RT; j++) xb[j] = *reinterpret_cast<const bf16x8 *>(&sX[b][(wave >> 1) * 32 * RT + 32 * j + m][16 * u + 8 * kg]);
#pragma unroll
            for (int i = 0; i < RN; i++)
#pragma unroll
                for (int j = 0; j < RT; j++) {
                    acc[i][j] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(wa[i], xb[j], acc[i][j], 0, 0, 0);
                    if (GATED) acc2[i][j] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(wb[i], xb[j], acc2[i][j], 0, 0, 0);
                }
        }
    };
    const auto each_set = [&](auto f) {                         // f(0), f(1), .. until one says stop
        if (!f(std::integral_constant<int, 0>()) || !f(std::integral_constant<int, 1>())) return false;
        if constexpr (SETS == 4) return f(std::integral_constant<int, 2>()) && f(std::integral_constant<int, 3>());
        return true;
    };
    each_set([&](auto set) { request(set, decltype(set)::value * MMT_K); return true; });   // (a stage past K is all zeros)
    for (int k0 = 0; k0 < a.K; k0 += SETS * MMT_K) {
        if (!each_set([&](auto set) {
                const int k = k0 + decltype(set)::value * MMT_K;
                if (k >= a.K) return false;
                stage(set);
                if (k + SETS * MMT_K < a.K) request(set, k + SETS * MMT_K);
                __syncthreads();
                multiply(set);
                return true;
            })) break;
    }
    // register r of a lane: weight row (r & 3) + 8 (r >> 2) + 4 kg of the tile, token = lane & 31
#pragma unroll
    for (int j = 0; j < RT; j++) {
        const int t = t0 + (wave >> 1) * 32 * RT + 32 * j + m;
        if (t >= v.rows) continue;
        const size_t yr = y_row(a, v, t);
        const float rs = a.row_scale ? a.row_scale[v.y0 + t] : 1.0f;
#pragma unroll
        for (int i = 0; i < RN; i++)
#pragma unroll
            for (int r = 0; r < 16; r++) {
                const int n = n0 + (wave & 1) * 32 * RN + 32 * i + (r & 3) + 8 * (r >> 2) + 4 * kg;
                if (n < a.N) y_store<EPI>(a, v, yr, n, acc[i][j][r], GATED ? acc2[i][j][r] : 0.0f, rs, v.resid ? v.resid[yr + n] : 0.0f);
            }
    }
}

template <int RN, int RT, int EPI>
static hipError_t launch_mmb_mfma(const MMBArgs &a, int rows_max, hipStream_t st) {
    const int nt = (a.N + 64 * RN - 1) / (64 * RN), tt = (rows_max + 64 * RT - 1) / (64 * RT);
    hipLaunchKernelGGL((mmb_mfma_kernel<RN, RT, EPI>), dim3((unsigned)((nt + 7) / 8 * 8 * tt), 1, (unsigned)a.nz), dim3(256), 0, st, a, nt, tt);
    return hipGetLastError();
}
// the tile by what a stage costs a CU in bytes fetched (KB: weights 8 per 64 rows and set, X 16 per 64 rows) times the rounds of workgroups the device needs; a
// grouped batch sizes its grid for the most rows ONE expert could hold, what counts is the rows an expert holds on average
template <int EPI>
static hipError_t launch_mmb_mfma_tile(const MMBArgs &a, int rows_max, hipStream_t st) {
    const long long rows = a.meta ? (a.T + a.nz - 1) / a.nz : rows_max;
    const auto rounds = [&](int rn, int rt, int kb) {
        const double wg = (double)((a.N + 64 * rn - 1) / (64 * rn)) * (double)((rows + 64 * rt - 1) / (64 * rt)) * a.nz;
        return (wg > 256.0 ? wg / 256.0 : 1.0) * kb;
    };
    if (EPI >= MMB_SILU_MUL) return rounds(1, 2, 48) < rounds(1, 1, 32) ? launch_mmb_mfma<1, 2, EPI>(a, rows_max, st) : launch_mmb_mfma<1, 1, EPI>(a, rows_max, st);
    const double r11 = rounds(1, 1, 24), r21 = rounds(2, 1, 32), r22 = rounds(2, 2, 48);
    if (r22 <= r11 && r22 <= r21) return launch_mmb_mfma<(EPI >= MMB_SILU_MUL ? 1 : 2), (EPI >= MMB_SILU_MUL ? 1 : 2), EPI>(a, rows_max, st);
    return r21 <= r11 ? launch_mmb_mfma<(EPI >= MMB_SILU_MUL ? 1 : 2), 1, EPI>(a, rows_max, st) : launch_mmb_mfma<1, 1, EPI>(a, rows_max, st);
}
template <bool VEC, int TB>
static void launch_mmb_vec(const MMBArgs &a, dim3 grid, hipStream_t st) {
    constexpr bool one = TB == 1;                               // (the epilogue as an argument: single rows only)
    if (a.ln) {
        if (one && a.epi == MMB_STORE) hipLaunchKernelGGL((mmb_vec_kernel<VEC, TB, (one ? (int)MMB_STORE : EPI_ANY), true>), grid, dim3(256), 0, st, a);
        else if (one && a.epi == MMB_CLAMP_SWIGLU) hipLaunchKernelGGL((mmb_vec_kernel<VEC, TB, (one ? (int)MMB_CLAMP_SWIGLU : EPI_ANY), true>), grid, dim3(256), 0, st, a);
        else hipLaunchKernelGGL((mmb_vec_kernel<VEC, TB, EPI_ANY, true>), grid, dim3(256), 0, st, a);
    } else if (one && a.epi == MMB_STORE) hipLaunchKernelGGL((mmb_vec_kernel<VEC, TB, (one ? (int)MMB_STORE : EPI_ANY), false>), grid, dim3(256), 0, st, a);
    else if (one && a.epi == MMB_SILU_MUL) hipLaunchKernelGGL((mmb_vec_kernel<VEC, TB, (one ? (int)MMB_SILU_MUL : EPI_ANY), false>), grid, dim3(256), 0, st, a);
    else hipLaunchKernelGGL((mmb_vec_kernel<VEC, TB, EPI_ANY, false>), grid, dim3(256), 0, st, a);
}
template <bool LN>
static void launch_mmb_vec_rows(const MMBArgs &a, int rows_max, dim3 grid, hipStream_t st) {
    if (rows_max == 1 && a.epi == MMB_STORE) hipLaunchKernelGGL((mmb_vec_rows_kernel<4, 1, MMB_STORE, LN>), grid, dim3(256), 0, st, a);
    else if (rows_max == 1) hipLaunchKernelGGL((mmb_vec_rows_kernel<4, 1, EPI_ANY, LN>), grid, dim3(256), 0, st, a);
    else hipLaunchKernelGGL((mmb_vec_rows_kernel<4, 4, EPI_ANY, LN>), grid, dim3(256), 0, st, a);
}

}  // namespace

hipError_t launch_mmb(const MMBArgs &a, hipStream_t st) {
    if (a.T <= 0 || a.N <= 0 || a.nz <= 0) return hipSuccess;
    const bool gated = a.epi == MMB_SILU_MUL || a.epi == MMB_GELU_MUL || a.epi == MMB_CLAMP_SWIGLU;
    if (a.K <= 0 || !a.x || !a.w || !a.y || (gated && !a.w2) || (a.x_map && !a.meta) || (a.y_map && !a.meta)) return hipErrorInvalidValue;
    const auto al = [](const void *p, size_t n) { return (reinterpret_cast<uintptr_t>(p) & (n - 1)) == 0; };
    // 16-byte loads of both operands: every row start and every stride on a 16-byte boundary
    const bool vec = (a.K % 8) == 0 && (a.ldw % 8) == 0 && (a.w_zs % 8) == 0 && (a.ldx % 4) == 0 && (a.x_zs % 4) == 0 && al(a.w, 16) && al(a.x, 16) &&
                     (!a.w2 || al(a.w2, 16)) && (!a.pn_w || al(a.pn_w, 16));
    const int rows_max = a.sel ? 1 : a.T;                        // most rows any outer index can hold
    if (a.pn_w && rows_max > MMB_VEC_ROWS) return hipErrorInvalidValue;   // (the norm prologue lives in the few-rows kernel only)
    if (a.ln && (!a.pn_w || a.sel || a.meta || a.nz != 1 || (gated && !a.ln2))) return hipErrorInvalidValue;
    if (rows_max <= MMB_VEC_ROWS || a.sel) {
        const dim3 grid((unsigned)((a.N + 3) / 4), (unsigned)a.nz);
        // many columns, a handful of rows: four weight rows per wave (the grid still has thousands of waves)
        if (vec && !a.sel && !a.meta && rows_max <= 4 && (long long)a.N * a.nz >= 4096) {
            const dim3 g4((unsigned)((a.N + 15) / 16), (unsigned)a.nz);
            if (a.ln) launch_mmb_vec_rows<true>(a, rows_max, g4, st);
            else launch_mmb_vec_rows<false>(a, rows_max, g4, st);
            return hipGetLastError();
        }
        if (vec && rows_max == 1) launch_mmb_vec<true, 1>(a, grid, st);
        else if (vec) launch_mmb_vec<true, 8>(a, grid, st);
        else launch_mmb_vec<false, 8>(a, grid, st);
        return hipGetLastError();
    }
    if (!a.f32 && vec && (a.K % 16) == 0) {
        switch (a.epi) {
            case MMB_STORE: return launch_mmb_mfma_tile<MMB_STORE>(a, rows_max, st);
            case MMB_RELU2: return launch_mmb_mfma_tile<MMB_RELU2>(a, rows_max, st);
            case MMB_SILU_MUL: return launch_mmb_mfma_tile<MMB_SILU_MUL>(a, rows_max, st);
            case MMB_GELU_MUL: return launch_mmb_mfma_tile<MMB_GELU_MUL>(a, rows_max, st);
            case MMB_CLAMP_SWIGLU: return launch_mmb_mfma_tile<MMB_CLAMP_SWIGLU>(a, rows_max, st);
            default: return hipErrorInvalidValue;
        }
    }
    const dim3 grid((unsigned)((a.N + 63) / 64), (unsigned)((rows_max + 63) / 64), (unsigned)a.nz);
    if (gated) hipLaunchKernelGGL(mmb_f32_kernel<true>, grid, dim3(256), 0, st, a);
    else hipLaunchKernelGGL(mmb_f32_kernel<false>, grid, dim3(256), 0, st, a);
    return hipGetLastError();
}

}  // namespace mi355
