// Shared helpers of the kernels behind poptransformer_hybrid.h: element types and workgroup reductions.
#pragma once
#include "../common.h"
#include "../../../include/poptransformer_hybrid.h"

// Eight consecutive elements of a row as fp32.  `vec`: the address is 16-byte aligned and all eight exist; otherwise
// elements from `valid` on are zero.
__device__ __forceinline__ void load8(const bf16* p, bool vec, int valid, float (&v)[8]) {
  if (vec) {
    const bf16x8 b = *reinterpret_cast<const bf16x8*>(p);
#pragma unroll
    for (int e = 0; e < 8; ++e) v[e] = (float)b[e];
  } else {
#pragma unroll
    for (int e = 0; e < 8; ++e) v[e] = e < valid ? (float)p[e] : 0.f;
  }
}
__device__ __forceinline__ void load8(const float* p, bool vec, int valid, float (&v)[8]) {
  if (vec) {
    const f32x4 a = *reinterpret_cast<const f32x4*>(p), b = *reinterpret_cast<const f32x4*>(p + 4);
#pragma unroll
    for (int e = 0; e < 4; ++e) { v[e] = a[e]; v[4 + e] = b[e]; }
  } else {
#pragma unroll
    for (int e = 0; e < 8; ++e) v[e] = e < valid ? p[e] : 0.f;
  }
}
__device__ __forceinline__ void store8(bf16* p, const float (&v)[8]) {
  bf16x8 b;
#pragma unroll
  for (int e = 0; e < 8; ++e) b[e] = (bf16)v[e];
  *reinterpret_cast<bf16x8*>(p) = b;
}
__device__ __forceinline__ void store8(float* p, const float (&v)[8]) {
  *reinterpret_cast<f32x4*>(p) = f32x4{v[0], v[1], v[2], v[3]};
  *reinterpret_cast<f32x4*>(p + 4) = f32x4{v[4], v[5], v[6], v[7]};
}

__device__ __forceinline__ float sigmoid_f32(float z) { return 1.0f / (1.0f + expf(-z)); }

// Sum over a workgroup of WAVES waves, in every thread; `buf` holds WAVES floats and may be reused after the next barrier.
template <int WAVES>
__device__ __forceinline__ float workgroup_sum(float v, float* buf) {
  v = wave_total_dpp(v);
  if ((threadIdx.x & 63) == 0) buf[threadIdx.x >> 6] = v;
  __syncthreads();
  float t = 0.f;
#pragma unroll
  for (int w = 0; w < WAVES; ++w) t += buf[w];
  return t;
}
