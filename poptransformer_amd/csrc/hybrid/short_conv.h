// Short causal convolutions: what the kernels that convolve share.  The ring of a slot keeps a sequence's newest rows as they came
// from the projection, position p in row p % taps: a row's own place is none of those it reads.
#pragma once
#include "attention.h"

// silu in fp32; for results that are rounded to bf16 by the hardware's exponential and reciprocal (a few units in the last place)
template <typename T> __device__ __forceinline__ float silu_of(float z);
template <> __device__ __forceinline__ float silu_of<float>(float z) { return z / (1.0f + expf(-z)); }
template <> __device__ __forceinline__ float silu_of<bf16>(float z) { return z * __builtin_amdgcn_rcpf(1.0f + __expf(-z)); }

// eight channels of position p as the ring holds them (zeros before the start)
template <typename T>
__device__ __forceinline__ void conv_ring8(const T* ring, int channels, int taps, int p, float (&v)[8]) {
  load8(ring + (size_t)((unsigned)(p > 0 ? p : 0) % (unsigned)taps) * channels, true, 8, v);
#pragma unroll
  for (int e = 0; e < 8; ++e) v[e] = p >= 0 ? v[e] : 0.f;
}

// Eight channels from c0 on of one row at position pos: v holds the row's own values and becomes the rounded result.
// What the three rows before it need is requested at once.
template <typename T>
__device__ __forceinline__ void conv8(const pta_conv& c, int slot, int pos, int c0, float (&v)[8]) {
  constexpr int NEAR = 3;
  const T* ring = reinterpret_cast<const T*>(c.ring) + (size_t)slot * c.taps * c.channels + c0;
  const float* weight = c.weight + c0;
  const int own = (int)((unsigned)pos % (unsigned)c.taps);
  float s[8], w[NEAR + 1][8];
  Raw8<T> u[NEAR + 1];
  load8(c.bias ? c.bias + c0 : nullptr, c.bias != nullptr, 0, s);
  load8(weight + (size_t)(c.taps - 1) * c.channels, true, 8, w[0]);
#pragma unroll
  for (int b = 1; b <= NEAR; ++b) {
    const int back = b < c.taps ? b : 0, row = own - back;
    u[b].load(ring + (size_t)(row < 0 ? row + c.taps : row) * c.channels, true, 8);
    load8(weight + (size_t)(c.taps - 1 - back) * c.channels, true, 8, w[b]);
  }
  for (int back = c.taps - 1; back > NEAR; --back) {
    float x[8], f[8];
    conv_ring8(ring, c.channels, c.taps, pos - back, x);
    load8(weight + (size_t)(c.taps - 1 - back) * c.channels, true, 8, f);
#pragma unroll
    for (int e = 0; e < 8; ++e) s[e] = __builtin_fmaf(f[e], x[e], s[e]);
  }
#pragma unroll
  for (int b = NEAR; b >= 1; --b) {
    float x[8];
    u[b].unpack(x);
    const bool there = b < c.taps && b <= pos;
#pragma unroll
    for (int e = 0; e < 8; ++e) s[e] = __builtin_fmaf(there ? w[b][e] : 0.f, there ? x[e] : 0.f, s[e]);
  }
#pragma unroll
  for (int e = 0; e < 8; ++e) {
    s[e] = __builtin_fmaf(w[0][e], v[e], s[e]);
    v[e] = (float)(T)(c.silu ? silu_of<T>(s[e]) : s[e]);
  }
}

// the place of position pos in the ring, from channel c0 on
template <typename T>
__device__ __forceinline__ T* conv_place(const pta_conv& c, int slot, int pos, int c0) {
  return reinterpret_cast<T*>(c.ring) + ((size_t)slot * c.taps + (unsigned)pos % (unsigned)c.taps) * c.channels + c0;
}

static inline int check_conv(const pta_conv& c, const char* name) {
  PTA_REQUIRE(c.taps >= 1 && c.taps <= PTA_CONV_TILE && c.channels > 0 && c.channels % 8 == 0, "%s: %d taps (1 .. %d) of %d channels (a multiple of 8)",
              name, c.taps, (int)PTA_CONV_TILE, c.channels);
  PTA_REQUIRE(c.weight && c.ring && pta_aligned(c.weight, 16) && pta_aligned(c.ring, 16) && pta_aligned(c.bias, 16), "%s: null or unaligned convolution", name);
  return PTA_OK;
}
