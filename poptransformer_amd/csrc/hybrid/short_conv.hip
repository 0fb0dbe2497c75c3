// Causal convolutions over a few tokens, channel by channel: the rows of a pass.  (Passes of single rows do this within the launch
// that reads the result, with conv8 of short_conv.h.)
#include "short_conv.h"

typedef pta_short_conv_args SC;

constexpr int SC_ROWS = 16;              // rows a wave walks through

// A wave takes eight channels per lane of `each` rows of a tile.  TAPS > 0: the rows before stay in registers.  The wave that holds a
// sequence's first row of the pass is the only one that reads the ring, and the one that leaves the sequence's newest rows there.
template <typename T, int TAPS>
__global__ __launch_bounds__(64) void short_conv_kernel(SC a, int each, int parts) {
  const int tile = blockIdx.x / parts, skip = (blockIdx.x % parts) * each;
  const int row0 = a.tile_row[tile], count = a.tile_count[tile];
  const int c0 = (blockIdx.y * 64 + threadIdx.x) * 8;
  if (skip >= count || c0 >= a.c.channels) return;
  const int r0 = row0 + skip, r1 = row0 + (skip + each < count ? skip + each : count);
  const int taps = TAPS > 0 ? TAPS : a.c.taps;
  const int last = skip == 0 ? a.last[row0] : -1;             // >= 0: r0 is its sequence's first row
  const int slot = a.slot[r0], p0 = a.pos[r0];
  const T* x = reinterpret_cast<const T*>(a.x) + c0;
  T* y = reinterpret_cast<T*>(a.y) + c0;
  T* ring = reinterpret_cast<T*>(a.c.ring) + (size_t)slot * taps * a.c.channels + c0;
  // the row `back` rows before r
  auto before = [&](int r, int back, float (&v)[8]) {
    if (last < 0 || r - back >= r0) load8(x + (size_t)(r - back) * a.ld_x, true, 8, v);
    else conv_ring8(ring, a.c.channels, taps, p0 + (r - r0) - back, v);
  };
  float bias[8];
  load8(a.c.bias ? a.c.bias + c0 : nullptr, a.c.bias != nullptr, 0, bias);
  auto put = [&](int r, float (&s)[8]) {
    if (a.c.silu)
#pragma unroll
      for (int e = 0; e < 8; ++e) s[e] = silu_of<T>(s[e]);
    store8(y + (size_t)r * a.ld_y, s);
  };
  if constexpr (TAPS > 0) {
    float w[TAPS][8], u[TAPS][8];                             // u[j]: the row TAPS - 1 - j before the current one
#pragma unroll
    for (int j = 0; j < TAPS; ++j) {
      load8(a.c.weight + (size_t)j * a.c.channels + c0, true, 8, w[j]);
      if (j > 0) before(r0, TAPS - j, u[j]);
    }
    constexpr int AHEAD = 4;                                  // rows requested together
    Raw8<T> next[AHEAD];
    auto fetch = [&](int r) {
#pragma unroll
      for (int k = 0; k < AHEAD; ++k) next[k].load(x + (size_t)(r + k < r1 ? r + k : r1 - 1) * a.ld_x, true, 8);
    };
    fetch(r0);
    for (int r = r0; r < r1; r += AHEAD) {
      Raw8<T> now[AHEAD];
#pragma unroll
      for (int k = 0; k < AHEAD; ++k) now[k] = next[k];
      fetch(r + AHEAD < r1 ? r + AHEAD : r);
#pragma unroll
      for (int k = 0; k < AHEAD; ++k) {
        if (r + k >= r1) break;
#pragma unroll
        for (int j = 0; j + 1 < TAPS; ++j)
#pragma unroll
          for (int e = 0; e < 8; ++e) u[j][e] = u[j + 1][e];
        now[k].unpack(u[TAPS - 1]);
        float s[8];
#pragma unroll
        for (int e = 0; e < 8; ++e) {
          s[e] = bias[e];
#pragma unroll
          for (int j = 0; j < TAPS; ++j) s[e] = __builtin_fmaf(w[j][e], u[j][e], s[e]);
        }
        put(r + k, s);
      }
    }
  } else {
    for (int r = r0; r < r1; ++r) {
      float s[8], u[8], w[8];
#pragma unroll
      for (int e = 0; e < 8; ++e) s[e] = bias[e];
      for (int j = 0; j < taps; ++j) {
        before(r, taps - 1 - j, u);
        load8(a.c.weight + (size_t)j * a.c.channels + c0, true, 8, w);
#pragma unroll
        for (int e = 0; e < 8; ++e) s[e] = __builtin_fmaf(w[e], u[e], s[e]);
      }
      put(r, s);
    }
  }
  if (last < 0) return;
  for (int r = last - taps + 1 > r0 ? last - taps + 1 : r0; r <= last; ++r) {
    float v[8];
    load8(x + (size_t)r * a.ld_x, true, 8, v);
    store8(ring + (size_t)((unsigned)(p0 + r - r0) % (unsigned)taps) * a.c.channels, v);
  }
}

extern "C" int pta_short_conv(const SC* args, pta_stream_t stream) {
  const char* name = "pta_short_conv";
  PTA_REQUIRE(args, "%s: null arguments", name);
  const SC& a = *args;
  PTA_REQUIRE(a.dtype == PTA_BF16 || a.dtype == PTA_FP32, "%s: unknown type %d", name, a.dtype);
  const int rc = check_conv(a.c, name);
  if (rc) return rc;
  PTA_REQUIRE(a.x && a.y && a.x != a.y && pta_aligned(a.x, 16) && pta_aligned(a.y, 16) && a.ld_x % 8 == 0 && a.ld_y % 8 == 0 &&
              a.ld_x >= a.c.channels && a.ld_y >= a.c.channels, "%s: null or unaligned rows (of %d and %d)", name, a.ld_x, a.ld_y);
  PTA_REQUIRE(a.slot && a.pos && a.last && a.tile_row && a.tile_count && a.tiles > 0, "%s: the rows' places are missing, or %d tiles", name, a.tiles);
  // only a sequence's first wave looks into the ring, so the others have to find every row they need among the pass's
  const int each = a.c.taps - 1 <= SC_ROWS ? SC_ROWS : (a.c.taps + 15) / 16 * 16, parts = (PTA_CONV_TILE + each - 1) / each;
  const dim3 grid((unsigned)(a.tiles * parts), (a.c.channels + 511) / 512);
  hipStream_t s = (hipStream_t)stream;
  auto launch = [&](auto taps) {
    constexpr int N = decltype(taps)::value;
    if (a.dtype == PTA_BF16) hipLaunchKernelGGL((short_conv_kernel<bf16, N>), grid, dim3(64), 0, s, a, each, parts);
    else hipLaunchKernelGGL((short_conv_kernel<float, N>), grid, dim3(64), 0, s, a, each, parts);
  };
  switch (a.c.taps) {
    case 1: launch(std::integral_constant<int, 1>{}); break;
    case 2: launch(std::integral_constant<int, 2>{}); break;
    case 3: launch(std::integral_constant<int, 3>{}); break;
    case 4: launch(std::integral_constant<int, 4>{}); break;
    default: launch(std::integral_constant<int, 0>{});
  }
  PTA_CHECK_LAUNCH(name);
  return PTA_OK;
}
