// attn_merge_dev.h — joining the records of an attention scan that was cut into runs of cells: record s = [maximum | sum | n weighted values] of run s.
// A workgroup of 256 threads per (row, head): lane s of every wave holds run s's maximum and sum (one trip to memory for all runs), then thread = value column.
#pragma once

#include <hip/hip_runtime.h>

namespace mi355 {

constexpr int ATTN_MERGE_MAX_RUNS = 64;

// sums[i] (LDS, n floats) = sum over the runs of e^(maximum_s - M) * value_s[i]; returns the softmax denominator under M = the maximum of all runs and of the
// sink (sink = -inf: none).  part: max(n, 256) floats of LDS; the caller reads sums behind the barrier this function ends with.
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
    // columns side by side as far as they go; narrow records share the runs among 2 or 4 groups of threads, whose sums meet in LDS
    const int groups = n <= 64 ? 4 : n <= 128 ? 2 : 1, width = 256 / groups, grp = tid / width;
    for (int i = tid - grp * width; i < n; i += width) {
        float o = 0.0f;
#pragma unroll 8
        for (int s = grp; s < splits; s += groups) { const float v = rec[(size_t)s * stride + 2 + i]; o += fac[s] > 0.0f ? v * fac[s] : 0.0f; }
        part[grp * n + i] = o;
    }
    __syncthreads();
    for (int i = tid; i < n; i += 256) sums[i] = groups == 1 ? part[i] : groups == 2 ? part[i] + part[n + i] : (part[i] + part[n + i]) + (part[2 * n + i] + part[3 * n + i]);
    __syncthreads();
    return den;
}

}  // namespace mi355
