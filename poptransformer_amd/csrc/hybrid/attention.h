// Helpers of the attention kernels behind poptransformer_hybrid.h.
#pragma once
#include "hybrid.h"
#include <type_traits>

template <typename T> __device__ __forceinline__ float exp_of(float x);
template <> __device__ __forceinline__ float exp_of<float>(float x) { return expf(x); }
template <> __device__ __forceinline__ float exp_of<bf16>(float x) { return __expf(x); }

// Sum over each group of L consecutive lanes, in every lane of the group (all lanes active).
template <int L>
__device__ __forceinline__ float group_sum(float v) {
  auto dpp = [](float x, auto ctrl) {
    return __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, x), decltype(ctrl)::value, 0xF, 0xF, true));
  };
  if (L >= 2) v += dpp(v, std::integral_constant<int, 0xB1>{});       // quad_perm [1, 0, 3, 2]
  if (L >= 4) v += dpp(v, std::integral_constant<int, 0x4E>{});       // quad_perm [2, 3, 0, 1]
  if (L >= 8) v += dpp(v, std::integral_constant<int, 0x141>{});      // row_half_mirror
  if (L >= 16) v += dpp(v, std::integral_constant<int, 0x140>{});     // row_mirror
  if (L >= 32) v += __shfl_xor(v, 16, 64);
  if (L >= 64) v += __shfl_xor(v, 32, 64);
  return v;
}

// eight elements on their way from memory
template <typename T> struct Raw8;
template <> struct Raw8<bf16> {
  u32x4 w;
  __device__ __forceinline__ void load(const bf16* p, bool vec, int valid) {
    if (vec) {
      w = *reinterpret_cast<const u32x4*>(p);
    } else {
      bf16x8 z;
#pragma unroll
      for (int e = 0; e < 8; ++e) z[e] = e < valid ? p[e] : (bf16)0.0f;
      w = bitcast<u32x4>(z);
    }
  }
  __device__ __forceinline__ void unpack(float (&v)[8]) const {
#pragma unroll
    for (int e = 0; e < 4; ++e) { v[2 * e] = bitcast<float>(w[e] << 16); v[2 * e + 1] = bitcast<float>(w[e] & 0xffff0000u); }
  }
};
template <> struct Raw8<float> {
  float w[8];
  __device__ __forceinline__ void load(const float* p, bool vec, int valid) { load8(p, vec, valid, w); }
  __device__ __forceinline__ void unpack(float (&v)[8]) const {
#pragma unroll
    for (int e = 0; e < 8; ++e) v[e] = w[e];
  }
};

typedef short s16x4 __attribute__((ext_vector_type(4)));

__device__ __forceinline__ f32x4 mma(bf16x8 a, bf16x8 b, f32x4 c) { return __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, c, 0, 0, 0); }

// Transposed read of a row-major LDS tile: of the 16 lanes of a group, lane i gives the address of four elements of row i / 4
// (columns 4 (i % 4) ..) and gets column i of the four rows.
__device__ __forceinline__ bf16x4 read_transposed(const bf16* p) {
  return bitcast<bf16x4>(__builtin_amdgcn_ds_read_tr16_b64_v4i16((__attribute__((address_space(3))) s16x4*)p));
}
__device__ __forceinline__ bf16x8 join(bf16x4 lo, bf16x4 hi) { return __builtin_shufflevector(lo, hi, 0, 1, 2, 3, 4, 5, 6, 7); }

// eight features from f on (f a multiple of eight) of a rotated part, turned by the row's angles
__device__ __forceinline__ void rotate8(const float* cs, float (&v)[8]) {
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const float c = cs[2 * i], s = cs[2 * i + 1], x = v[2 * i], y = v[2 * i + 1];
    v[2 * i] = x * c - y * s;
    v[2 * i + 1] = y * c + x * s;
  }
}
