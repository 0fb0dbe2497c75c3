// A residual that takes normed results: x <- x + rms_norm(y) * weight, with what follows in the same launch: the rounded row that
// the next sublayer reads, or the model's norm of it, and the routing of the row to its experts.
#include "attention.h"
#include "routing.h"

typedef pta_result_norm_args RN;

// Many rows (bf16): sixteen of them per workgroup, whose waves share the features; BLOCKS * 16 logits of each at a time.
constexpr int RR_WAVES = 8;

template <int BLOCKS>
__global__ __launch_bounds__(RR_WAVES * 64) void route_rows_kernel(const bf16* h, int ld, int rows, const bf16x8* router, pta_routing g, int z_ld) {
  extern __shared__ __align__(16) float z_rows[];            // [16][z_ld]
  __shared__ f32x4 red[RR_WAVES][BLOCKS][64];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, lg = lane >> 4, lc = lane & 15;
  const int row0 = blockIdx.x * 16, n = g.experts + g.shared, pieces = (ld + 127) / 128 * 4, last = (n + 15) / 16 - 1;
  const bf16* x = h + (size_t)(row0 + lc < rows ? row0 + lc : rows - 1) * ld;
  for (int e0 = 0; e0 < n; e0 += BLOCKS * 16) {
    const bf16x8* w[BLOCKS];
    f32x4 acc[BLOCKS];
#pragma unroll
    for (int b = 0; b < BLOCKS; ++b) {
      w[b] = router + (size_t)(e0 / 16 + b < last ? e0 / 16 + b : last) * pieces * 64 + lane;
      acc[b] = f32x4{0.f, 0.f, 0.f, 0.f};
    }
    const int per = (pieces + RR_WAVES - 1) / RR_WAVES, end = (wave + 1) * per < pieces ? (wave + 1) * per : pieces;
    constexpr int U = 4;                                     // pieces whose operands are requested together
    for (int c0 = wave * per; c0 < end; c0 += U) {
      bf16x8 xv[U], wv[U][BLOCKS];
#pragma unroll
      for (int u = 0; u < U; ++u) {
        const int c = c0 + u < end ? c0 + u : end - 1, k = c * 32 + lg * 8;
        xv[u] = *reinterpret_cast<const bf16x8*>(x + (k < ld ? k : 0));
#pragma unroll
        for (int b = 0; b < BLOCKS; ++b) wv[u][b] = w[b][(size_t)c * 64];
      }
      __builtin_amdgcn_sched_barrier(0);
#pragma unroll
      for (int u = 0; u < U; ++u) {
        const bool in = c0 + u < end && (c0 + u) * 32 + lg * 8 < ld;
#pragma unroll
        for (int i = 0; i < 8; ++i) xv[u][i] = in ? xv[u][i] : (bf16)0.0f;
#pragma unroll
        for (int b = 0; b < BLOCKS; ++b) acc[b] = mma(wv[u][b], xv[u], acc[b]);
      }
    }
    __syncthreads();
#pragma unroll
    for (int b = 0; b < BLOCKS; ++b) red[wave][b][lane] = acc[b];
    __syncthreads();
    for (int i = threadIdx.x; i < BLOCKS * 64; i += RR_WAVES * 64) {
      f32x4 s = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int v = 0; v < RR_WAVES; ++v) s += red[v][i / 64][i % 64];
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int e = e0 + i / 64 * 16 + i % 64 / 16 * 4 + r;
        if (e < n) z_rows[(i & 15) * z_ld + e] = s[r];
      }
    }
  }
  __syncthreads();
  for (int m = wave; m < 16; m += RR_WAVES) route_row<64>(g, z_rows + m * z_ld, row0 + m, lane, row0 + m < rows);
}

template <int PER>
__global__ __launch_bounds__(64) void route_kernel(const float* logits, pta_routing g) {
  __shared__ float z[ROUTE_FLOATS];
  const int n = g.experts + g.shared;
  for (int c = threadIdx.x; c < n; c += 64) z[c] = logits[(size_t)blockIdx.x * n + c];
  __syncthreads();
  route_row<64, PER>(g, z, blockIdx.x, threadIdx.x, true);
}

__device__ __forceinline__ float rounded(float v, bf16) { return (float)(bf16)v; }
__device__ __forceinline__ float rounded(float v, float) { return v; }

// One workgroup per row; a thread owns the columns c, c + 4 * THREADS, ... (four at a time) from the result to h.
template <typename T, int THREADS>
__global__ __launch_bounds__(THREADS) void result_norm_kernel(RN a) {
  constexpr int WAVES = THREADS / 64;
  extern __shared__ __align__(16) float u_row[];             // the result, then what h holds
  __shared__ float red[2][WAVES];
  __shared__ float z[ROUTE_FLOATS];
  __shared__ float pw[64];
  const int r = blockIdx.x, d = a.width;
  float* x = a.x + (size_t)r * d;
  T* h = reinterpret_cast<T*>(a.h) + (size_t)r * a.h_ld;
  const bool vec = (d & 3) == 0;
  const int step = vec ? THREADS * 4 : THREADS, span = vec ? 4 : 1;
  const T* row = nullptr;
  if (a.table) {
    int col = a.ids_index ? *a.ids_index : 0;
    col = col < 0 ? 0 : (col >= a.ids_stride ? a.ids_stride - 1 : col);
    int id = a.ids[(size_t)r * a.ids_stride + col];
    id = id < 0 ? 0 : (id >= a.vocab ? a.vocab - 1 : id);
    row = reinterpret_cast<const T*>(a.table) + (size_t)id * d;
    if (a.pos_out && threadIdx.x == 0) a.pos_out[r] = a.ids_index ? *a.ids_index : 0;
  }
  float inv = 0.f;
  if (!row) {
    const float* y = a.y ? a.y + (size_t)r * d : nullptr;
    const float yw = a.y && a.y_weight ? a.y_weight[(size_t)r * a.weights_ld] : 1.0f;
    if (a.parts) {
      if ((int)threadIdx.x < a.n_parts) pw[threadIdx.x] = a.part_weight[(size_t)r * a.weights_ld + threadIdx.x];
      __syncthreads();
    }
    float sq = 0.f;
    auto column = [&](auto width_tag, int c) {
      constexpr int V = decltype(width_tag)::value;
      float u[V] = {};
      if (y) {
        if constexpr (V == 4) {
          const f32x4 t = *reinterpret_cast<const f32x4*>(y + c);
#pragma unroll
          for (int e = 0; e < 4; ++e) u[e] = t[e] * yw;
        } else {
          u[0] = y[c] * yw;
        }
      }
      if (a.parts) {
        const size_t at = (size_t)r * a.parts_ld * d + c;
#pragma unroll 4
        for (int p = 0; p < a.n_parts; ++p) {
          float t[V];
          if (a.part_f32) {
            const float* s = reinterpret_cast<const float*>(a.parts) + at + (size_t)p * d;
            if constexpr (V == 4) {
              const f32x4 q = *reinterpret_cast<const f32x4*>(s);
#pragma unroll
              for (int e = 0; e < 4; ++e) t[e] = q[e];
            } else t[0] = s[0];
          } else {
            const T* s = reinterpret_cast<const T*>(a.parts) + at + (size_t)p * d;
            if constexpr (V == 4 && sizeof(T) == 2) {
              const bf16x4 q = *reinterpret_cast<const bf16x4*>(s);
#pragma unroll
              for (int e = 0; e < 4; ++e) t[e] = (float)q[e];
            } else {
#pragma unroll
              for (int e = 0; e < V; ++e) t[e] = (float)s[e];
            }
          }
#pragma unroll
          for (int e = 0; e < V; ++e) u[e] = __builtin_fmaf(pw[p], t[e], u[e]);
        }
      }
#pragma unroll
      for (int e = 0; e < V; ++e) {
        u_row[c + e] = u[e];
        sq = __builtin_fmaf(u[e], u[e], sq);
      }
    };
    if (vec) for (int c = threadIdx.x * 4; c < d; c += step) column(std::integral_constant<int, 4>{}, c);
    else for (int c = threadIdx.x; c < d; c += step) column(std::integral_constant<int, 1>{}, c);
    inv = 1.0f / sqrtf(workgroup_sum<WAVES>(sq, red[0]) / (float)d + a.eps);
  }
  float sq = 0.f;
  auto update = [&](auto width_tag, int c) {
    constexpr int V = decltype(width_tag)::value;
    float v[V];
    if (row) {
#pragma unroll
      for (int e = 0; e < V; ++e) v[e] = (float)row[c + e] * a.embed_scale;
    } else if constexpr (V == 4) {
      const f32x4 t = *reinterpret_cast<const f32x4*>(x + c), w = *reinterpret_cast<const f32x4*>(a.weight + c);
#pragma unroll
      for (int e = 0; e < 4; ++e) v[e] = t[e] + u_row[c + e] * inv * w[e];
    } else {
      v[0] = x[c] + u_row[c] * inv * a.weight[c];
    }
    if constexpr (V == 4) *reinterpret_cast<f32x4*>(x + c) = f32x4{v[0], v[1], v[2], v[3]};
    else x[c] = v[0];
#pragma unroll
    for (int e = 0; e < V; ++e) {
      u_row[c + e] = a.final_weight ? v[e] : rounded(v[e], T{});
      sq = __builtin_fmaf(v[e], v[e], sq);
    }
    if (!a.final_weight) {
      if constexpr (V == 4 && sizeof(T) == 2) {
        if ((a.h_ld & 3) == 0) {
          bf16x4 o;
#pragma unroll
          for (int e = 0; e < 4; ++e) o[e] = (bf16)v[e];
          *reinterpret_cast<bf16x4*>(h + c) = o;
          return;
        }
      }
#pragma unroll
      for (int e = 0; e < V; ++e) h[c + e] = (T)v[e];
    }
  };
  if (vec) for (int c = threadIdx.x * 4; c < d; c += step) update(std::integral_constant<int, 4>{}, c);
  else for (int c = threadIdx.x; c < d; c += step) update(std::integral_constant<int, 1>{}, c);
  if (a.final_weight) {
    const float f = 1.0f / sqrtf(workgroup_sum<WAVES>(sq, red[1]) / (float)d + a.eps);
    for (int c = threadIdx.x * span; c < d; c += step)
      for (int e = 0; e < span; ++e) h[c + e] = (T)(u_row[c + e] * f * a.final_weight[c + e]);
  }
  for (int c = d + threadIdx.x; c < a.h_ld; c += THREADS) h[c] = (T)0.0f;
  if (!a.router) return;
  router_logits<T, WAVES>(a.router, a.h_ld, d, u_row, a.routing, z);
  route_row<THREADS>(a.routing, z, r, threadIdx.x, true);
}

extern "C" int pta_route(const float* logits, int rows, const pta_routing* routing, pta_stream_t stream) {
  PTA_REQUIRE(logits && routing && rows > 0, "pta_route: null pointer, or %d rows", rows);
  const int rc = check_routing(*routing, "pta_route");
  if (rc) return rc;
  hipStream_t s = (hipStream_t)stream;
  if (routing->experts <= 64) hipLaunchKernelGGL((route_kernel<1>), dim3(rows), dim3(64), 0, s, logits, *routing);
  else if (routing->experts <= 256) hipLaunchKernelGGL((route_kernel<4>), dim3(rows), dim3(64), 0, s, logits, *routing);
  else hipLaunchKernelGGL((route_kernel<16>), dim3(rows), dim3(64), 0, s, logits, *routing);
  PTA_CHECK_LAUNCH("pta_route");
  return PTA_OK;
}

extern "C" int pta_route_rows(const uint16_t* h, int ld, int rows, const void* router, const pta_routing* routing, pta_stream_t stream) {
  const char* name = "pta_route_rows";
  PTA_REQUIRE(h && router && routing && rows > 0, "%s: null pointer, or %d rows", name, rows);
  PTA_REQUIRE(ld > 0 && ld % 8 == 0 && pta_aligned(h, 16) && pta_aligned(router, 16), "%s: rows of %d, or unaligned operands", name, ld);
  const int rc = check_routing(*routing, name);
  if (rc) return rc;
  const int z_ld = route_floats(*routing);
  const size_t smem = (size_t)16 * z_ld * sizeof(float);
  auto launch = [&](auto blocks) {
    constexpr int B = decltype(blocks)::value;
    PTA_REQUIRE(smem <= 24 * 1024 || hipFuncSetAttribute((const void*)route_rows_kernel<B>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)smem) ==
                                         hipSuccess, "%s: %zu bytes of LDS refused", name, smem);
    hipLaunchKernelGGL((route_rows_kernel<B>), dim3((rows + 15) / 16), dim3(RR_WAVES * 64), smem, (hipStream_t)stream,
                       reinterpret_cast<const bf16*>(h), ld, rows, reinterpret_cast<const bf16x8*>(router), *routing, z_ld);
    return PTA_OK;
  };
  const int blocks = (routing->experts + routing->shared + 15) / 16;
  const int launched = blocks == 1   ? launch(std::integral_constant<int, 1>{})
                       : blocks == 2 ? launch(std::integral_constant<int, 2>{})
                       : blocks == 3 ? launch(std::integral_constant<int, 3>{})
                                     : launch(std::integral_constant<int, 4>{});
  if (launched) return launched;
  PTA_CHECK_LAUNCH(name);
  return PTA_OK;
}

extern "C" int pta_result_norm(const RN* args, pta_stream_t stream) {
  const char* name = "pta_result_norm";
  PTA_REQUIRE(args, "%s: null arguments", name);
  const RN& a = *args;
  PTA_REQUIRE(a.dtype == PTA_BF16 || a.dtype == PTA_FP32, "%s: unknown type %d", name, a.dtype);
  PTA_REQUIRE(a.rows > 0 && a.width > 0 && a.width <= 14000, "%s: rows %d, width %d (1 .. 14000)", name, a.rows, a.width);
  PTA_REQUIRE(a.x && a.h && a.h_ld >= a.width && a.h_ld <= a.width + 7 && pta_aligned(a.x, 16) && pta_aligned(a.h, 16),
              "%s: x or h null or unaligned, h rows of %d", name, a.h_ld);
  PTA_REQUIRE(a.table ? (a.ids && a.vocab > 0 && a.ids_stride > 0 && !a.y && !a.parts) : ((a.y || a.parts) && a.weight),
              "%s: either an embedding with ids, or a result with its norm's weight", name);
  PTA_REQUIRE(pta_aligned(a.y, 16) && pta_aligned(a.parts, 16) && pta_aligned(a.weight, 16), "%s: unaligned result or weight", name);
  PTA_REQUIRE(!a.parts || (a.n_parts >= 1 && a.n_parts <= 64 && a.parts_ld >= a.n_parts && a.part_weight && a.weights_ld >= a.n_parts), "%s: %d parts (1 .. 64)", name, a.n_parts);
  PTA_REQUIRE(!a.y_weight || a.weights_ld >= 1, "%s: the weights' stride", name);
  if (a.router) {
    const int rc = check_routing(a.routing, name);
    if (rc) return rc;
    PTA_REQUIRE(!a.final_weight && a.h_ld % 8 == 0 && pta_aligned(a.router, 16), "%s: a router reads h, in whole pieces of eight", name);
  }
  hipStream_t s = (hipStream_t)stream;
  const size_t smem = (size_t)a.h_ld * sizeof(float);
  // few rows: a whole row of 1024 threads shortens the chain of a row; many rows: the machine is full either way
  const bool few = a.rows <= 64 && a.width >= 2048;
  auto launch = [&](auto threads) {
    constexpr int N = decltype(threads)::value;
    if (a.dtype == PTA_BF16) hipLaunchKernelGGL((result_norm_kernel<bf16, N>), dim3(a.rows), dim3(N), smem, s, a);
    else hipLaunchKernelGGL((result_norm_kernel<float, N>), dim3(a.rows), dim3(N), smem, s, a);
  };
  if (few) launch(std::integral_constant<int, 1024>{});
  else launch(std::integral_constant<int, 256>{});
  PTA_CHECK_LAUNCH(name);
  return PTA_OK;
}
