// attn_merge_dev.h — joining the records of an attention scan that was cut into runs of cells: record s = [maximum | sum | n weighted values] of run s.
// A workgroup of NT threads per (row, head) - many threads where few rows are joined and one trip to memory is all that counts -: lane s of every wave holds run s's maximum and sum (one trip to memory for all runs), then thread = value column.
#pragma once

#include <hip/hip_runtime.h>

namespace mi355 {

constexpr int ATTN_MERGE_MAX_RUNS = 64, ATTN_MERGE_FEW = 512;   // up to ATTN_MERGE_FEW (row, head) pairs are joined by 1024 threads each

// sums[i] (LDS, n floats) = sum over the runs of e^(maximum_s - M) * value_s[i]; returns the softmax denominator under M = the maximum of all runs and of the
// sink (sink = -inf: none).  part: max(NT / 256 * n, NT) floats of LDS; the caller reads sums behind the barrier this function ends with.
template <int NT>
__device__ __forceinline__ float attn_merge_runs(const float *rec, int splits, int n, float sink, float *fac, float *part, float *sums) {
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const size_t stride = (size_t)n + 2;
    float m = -INFINITY, l = 0.0f;
    if (lane < splits) { m = rec[(size_t)lane * stride]; l = rec[(size_t)lane * stride + 1]; }
    float M = fmaxf(l > 0.0f ? m : -INFINITY, sink);
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) M = fmaxf(M, __shfl_xor(M, o, 64));
    const float f = l > 0.0f ? expf(m - M) : 0.0f;
    float den = l * f;
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) den += __shfl_xor(den, o, 64);
    if (sink > -INFINITY) den += expf(sink - M);
    if (wave == 0) fac[lane] = f;
    __syncthreads();
    // columns side by side; groups of threads share the runs, their sums meet in LDS
    const int width = n <= 64 ? 64 : n <= 128 ? 128 : 256, groups = NT / width, grp = tid / width;
    for (int i = tid - grp * width; i < n; i += width) {
        float o = 0.0f;
#pragma unroll 8
        for (int s = grp; s < splits; s += groups) { const float v = rec[(size_t)s * stride + 2 + i]; o += fac[s] > 0.0f ? v * fac[s] : 0.0f; }
        part[grp * n + i] = o;
    }
    __syncthreads();
    for (int i = tid; i < n; i += NT) {
        float o = part[i];
        for (int g = 1; g < groups; g++) o += part[g * n + i];
        sums[i] = o;
    }
    __syncthreads();
    return den;
}

}  // namespace mi355
