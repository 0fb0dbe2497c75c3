// Next-token selection over fp32 logits: the largest entry of a row (ties: lowest index), or the k largest in order.
#include "hybrid.h"

constexpr int SEL_THREADS = 1024;

// (v, i) comes before (best, bi): larger value, or the same value at a lower index
__device__ __forceinline__ bool before(float v, int i, float best, int bi) { return v > best || (v == best && i < bi); }

// The k best entries, one pass over the row per pick: pass j takes the first entry, in that order, that comes after
// pick j - 1.  NaN compares false everywhere and is never picked; a row with nothing left gives index 0 and -inf.
__global__ __launch_bounds__(SEL_THREADS) void topk_f32_kernel(const float* __restrict__ x, int32_t* __restrict__ idx,
                                                               float* __restrict__ val, int n, int k) {
  __shared__ float sv[SEL_THREADS / 64];
  __shared__ int si[SEL_THREADS / 64];
  const float* row = x + (size_t)blockIdx.x * n;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  float last_v = INFINITY;
  int last_i = -1;
  for (int j = 0; j < k; ++j) {
    float best = -INFINITY;
    int bi = 0x7fffffff;
    for (int i = threadIdx.x; i < n; i += SEL_THREADS) {
      const float v = row[i];
      const bool left = v < last_v || (v == last_v && i > last_i);
      if (left && before(v, i, best, bi)) { best = v; bi = i; }
    }
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) {
      const float ov = __shfl_xor(best, o, 64);
      const int oi = __shfl_xor(bi, o, 64);
      if (before(ov, oi, best, bi)) { best = ov; bi = oi; }
    }
    if (lane == 0) { sv[wave] = best; si[wave] = bi; }
    __syncthreads();
    best = sv[0];
    bi = si[0];
    for (int w = 1; w < SEL_THREADS / 64; ++w)
      if (before(sv[w], si[w], best, bi)) { best = sv[w]; bi = si[w]; }
    if (threadIdx.x == 0) {
      idx[(size_t)blockIdx.x * k + j] = bi == 0x7fffffff ? 0 : bi;
      if (val) val[(size_t)blockIdx.x * k + j] = best;
    }
    last_v = best;
    last_i = bi;
    __syncthreads();
  }
}

// The best entry of a row: sixteen-byte loads, four of a thread's travelling together.
__global__ __launch_bounds__(SEL_THREADS) void argmax_f32_kernel(const float* __restrict__ x, int32_t* __restrict__ idx,
                                                                 float* __restrict__ val, int n, bool vec) {
  __shared__ float sv[SEL_THREADS / 64];
  __shared__ int si[SEL_THREADS / 64];
  const float* row = x + (size_t)blockIdx.x * n;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, nvec = vec ? n >> 2 : 0;
  float best = -INFINITY;
  int bi = 0x7fffffff;
  for (int c = threadIdx.x; c < nvec; c += 4 * SEL_THREADS) {
    f32x4 v[4];
#pragma unroll
    for (int u = 0; u < 4; ++u) {
      const int cu = c + u * SEL_THREADS;
      v[u] = *reinterpret_cast<const f32x4*>(row + (size_t)(cu < nvec ? cu : c) * 4);
    }
#pragma unroll
    for (int u = 0; u < 4; ++u) {
      const int cu = c + u * SEL_THREADS;
#pragma unroll
      for (int e = 0; e < 4; ++e)
        if (cu < nvec && before(v[u][e], cu * 4 + e, best, bi)) { best = v[u][e]; bi = cu * 4 + e; }
    }
  }
  for (int i = nvec * 4 + threadIdx.x; i < n; i += SEL_THREADS)
    if (before(row[i], i, best, bi)) { best = row[i]; bi = i; }
#pragma unroll
  for (int o = 32; o > 0; o >>= 1) {
    const float ov = __shfl_xor(best, o, 64);
    const int oi = __shfl_xor(bi, o, 64);
    if (before(ov, oi, best, bi)) { best = ov; bi = oi; }
  }
  if (lane == 0) { sv[wave] = best; si[wave] = bi; }
  __syncthreads();
  if (threadIdx.x == 0) {
    for (int w = 1; w < SEL_THREADS / 64; ++w)
      if (before(sv[w], si[w], best, bi)) { best = sv[w]; bi = si[w]; }
    idx[blockIdx.x] = bi == 0x7fffffff ? 0 : bi;
    if (val) val[blockIdx.x] = best;
  }
}

extern "C" int pta_topk_f32(const float* logits, int32_t* ids, float* values, int rows, int n, int k, pta_stream_t stream) {
  PTA_REQUIRE(logits && ids, "pta_topk_f32: null pointer");
  PTA_REQUIRE(rows > 0 && n > 0, "pta_topk_f32: empty input [%d,%d]", rows, n);
  PTA_REQUIRE(k >= 1 && k <= n, "pta_topk_f32: k must be in [1, %d], got %d", n, k);
  hipLaunchKernelGGL(topk_f32_kernel, dim3(rows), dim3(SEL_THREADS), 0, (hipStream_t)stream, logits, ids, values, n, k);
  PTA_CHECK_LAUNCH("pta_topk_f32");
  return PTA_OK;
}

extern "C" int pta_argmax_f32(const float* logits, int32_t* ids, float* values, int rows, int n, pta_stream_t stream) {
  PTA_REQUIRE(logits && ids, "pta_argmax_f32: null pointer");
  PTA_REQUIRE(rows > 0 && n > 0, "pta_argmax_f32: empty input [%d,%d]", rows, n);
  hipLaunchKernelGGL(argmax_f32_kernel, dim3(rows), dim3(SEL_THREADS), 0, (hipStream_t)stream, logits, ids, values, n,
                     n % 4 == 0 && pta_aligned(logits, 16));
  PTA_CHECK_LAUNCH("pta_argmax_f32");
  return PTA_OK;
}
