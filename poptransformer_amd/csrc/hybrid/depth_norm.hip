// The end of a layer whose result takes a normed addition and is then averaged with the residuals of all depths before it, with the
// next layer's norm and routing in the same launch; and the step before: a mixture's parts added to the residual.
#include "attention.h"
#include "routing.h"

typedef pta_depth_norm_args DN;

// One workgroup per row; a thread owns the columns c, c + 4 * THREADS, ... (four at a time) from the result to h.
template <typename T, int THREADS>
__global__ __launch_bounds__(THREADS) void depth_norm_kernel(DN a) {
  constexpr int WAVES = THREADS / 64;
  extern __shared__ __align__(16) float u_row[];             // the average, then what h holds
  __shared__ float red[3][WAVES];
  __shared__ float z[ROUTE_FLOATS];
  const int r = blockIdx.x, d = a.width;
  const bool vec = (d & 3) == 0;
  const int span = vec ? 4 : 1, step = THREADS * span, first = threadIdx.x * span;
  T* h = reinterpret_cast<T*>(a.h) + (size_t)r * a.h_ld;
  const float* base = a.history + (size_t)r * d;
  float* newest = a.history + (size_t)(a.depth > 0 ? a.depth - 1 : 0) * a.depth_stride + (size_t)r * d;
  float* next = a.next ? a.next + (size_t)r * d : nullptr;
  const float* y = a.y ? a.y + (size_t)r * d : nullptr;
  const T* row = nullptr;
  if (a.table) {
    int col = a.ids_index ? *a.ids_index : 0;
    col = col < 0 ? 0 : (col >= a.ids_stride ? a.ids_stride - 1 : col);
    int id = a.ids[(size_t)r * a.ids_stride + col];
    id = id < 0 ? 0 : (id >= a.vocab ? a.vocab - 1 : id);
    row = reinterpret_cast<const T*>(a.table) + (size_t)id * d;
    if (a.pos_out && threadIdx.x == 0) a.pos_out[r] = a.ids_index ? *a.ids_index : 0;
    if (a.side) {                                            // the token's parts of all layers, one behind the other
      const T* e = reinterpret_cast<const T*>(a.side_table) + (size_t)id * a.side_layers * a.side_ld;
      for (int c = threadIdx.x * 8; c < a.side_layers * a.side_ld; c += THREADS * 8) {
        float v[8];
        load8(e + c, true, 8, v);
        store8(reinterpret_cast<T*>(a.side) + (size_t)(c / a.side_ld) * a.side_stride + (size_t)r * a.side_ld + c % a.side_ld, v);
      }
    }
  }
  float inv = 0.f;
  if (y) {
    float sq = 0.f;
    if (vec) {
      for (int c = first; c < d; c += step) {
        const f32x4 t = *reinterpret_cast<const f32x4*>(y + c);
#pragma unroll
        for (int e = 0; e < 4; ++e) sq = __builtin_fmaf(t[e], t[e], sq);
      }
    } else {
      for (int c = first; c < d; c += step) sq = __builtin_fmaf(y[c], y[c], sq);
    }
    inv = 1.0f / sqrtf(workgroup_sum<WAVES>(sq, red[0]) / (float)d + a.eps);
  }
  float sum = 0.f;
  auto column = [&](auto width_tag, int c) {
    constexpr int V = decltype(width_tag)::value;
    auto load = [&](const float* p, float (&v)[V]) {
      if constexpr (V == 4) {
        const f32x4 t = *reinterpret_cast<const f32x4*>(p + c);
#pragma unroll
        for (int e = 0; e < 4; ++e) v[e] = t[e];
      } else {
        v[0] = p[c];
      }
    };
    auto store = [&](float* p, const float (&v)[V]) {
      if constexpr (V == 4) *reinterpret_cast<f32x4*>(p + c) = f32x4{v[0], v[1], v[2], v[3]};
      else p[c] = v[0];
    };
    float v[V], u[V] = {};
    if (row) {
#pragma unroll
      for (int e = 0; e < V; ++e) u[e] = (float)row[c + e] * a.embed_scale;
      store(newest, u);
    } else {
      load(newest, v);
      constexpr int AHEAD = 8;                               // depths requested together
      for (int j0 = 0; j0 < a.depth - 1; j0 += AHEAD) {
        float t[AHEAD][V];
#pragma unroll
        for (int j = 0; j < AHEAD; ++j) load(base + (size_t)(j0 + j < a.depth - 1 ? j0 + j : j0) * a.depth_stride, t[j]);
#pragma unroll
        for (int j = 0; j < AHEAD; ++j) {
          const float f = j0 + j < a.depth - 1 ? a.weights[j0 + j] : 0.f;
#pragma unroll
          for (int e = 0; e < V; ++e) u[e] = __builtin_fmaf(f, t[j][e], u[e]);
        }
      }
      if (y) {
        float t[V], w[V];
        load(y, t);
        load(a.y_weight, w);
#pragma unroll
        for (int e = 0; e < V; ++e) v[e] += t[e] * inv * w[e];
        store(newest, v);
      }
      const float f = a.weights ? a.weights[a.depth - 1] : 1.0f;
#pragma unroll
      for (int e = 0; e < V; ++e) u[e] = __builtin_fmaf(f, v[e], u[e]);
    }
    if (next) store(next, u);
#pragma unroll
    for (int e = 0; e < V; ++e) {
      u_row[c + e] = u[e];
      sum += u[e];
    }
  };
  if (vec) for (int c = first; c < d; c += step) column(std::integral_constant<int, 4>{}, c);
  else for (int c = first; c < d; c += step) column(std::integral_constant<int, 1>{}, c);
  const float mean = a.centred ? workgroup_sum<WAVES>(sum, red[1]) / (float)d : 0.f;
  float sq = 0.f;
  for (int c = first; c < d; c += step)
    for (int e = 0; e < span; ++e) {
      const float t = u_row[c + e] - mean;
      sq = __builtin_fmaf(t, t, sq);
    }
  const float f = 1.0f / sqrtf(workgroup_sum<WAVES>(sq, red[2]) / (float)d + a.eps);
  if (vec && (a.h_ld & 3) == 0) {
    typedef T vecT __attribute__((ext_vector_type(4)));
    for (int c = first; c < d; c += step) {
      const f32x4 u = *reinterpret_cast<const f32x4*>(u_row + c), w = *reinterpret_cast<const f32x4*>(a.norm_weight + c);
      vecT o;
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        o[e] = (T)((u[e] - mean) * f * w[e]);
        u_row[c + e] = (float)o[e];
      }
      *reinterpret_cast<vecT*>(h + c) = o;
    }
  } else {
    for (int c = first; c < d; c += step)
      for (int e = 0; e < span; ++e) {
        const T o = (T)((u_row[c + e] - mean) * f * a.norm_weight[c + e]);
        h[c + e] = o;
        u_row[c + e] = (float)o;
      }
  }
  for (int c = d + threadIdx.x; c < a.h_ld; c += THREADS) h[c] = (T)0.0f;
  if (!a.router) return;
  router_logits<T, WAVES>(a.router, a.h_ld, d, u_row, a.routing, z);
  route_row<THREADS>(a.routing, z, r, threadIdx.x, true);
}

extern "C" int pta_depth_norm(const DN* args, pta_stream_t stream) {
  const char* name = "pta_depth_norm";
  PTA_REQUIRE(args, "%s: null arguments", name);
  const DN& a = *args;
  PTA_REQUIRE(a.dtype == PTA_BF16 || a.dtype == PTA_FP32, "%s: unknown type %d", name, a.dtype);
  PTA_REQUIRE(a.rows > 0 && a.width > 0 && a.width <= 14000, "%s: rows %d, width %d (1 .. 14000)", name, a.rows, a.width);
  PTA_REQUIRE(a.history && pta_aligned(a.history, 16) && a.depth_stride >= (size_t)a.rows * a.width && a.depth_stride % 4 == 0 && pta_aligned(a.next, 16),
              "%s: the history is missing, unaligned, or too narrow", name);
  PTA_REQUIRE(a.h && pta_aligned(a.h, 16) && a.h_ld >= a.width && a.h_ld <= a.width + 7 && a.norm_weight && pta_aligned(a.norm_weight, 16),
              "%s: h or its norm's weight null or unaligned, h rows of %d", name, a.h_ld);
  PTA_REQUIRE(a.table ? (a.ids && a.vocab > 0 && a.ids_stride > 0 && a.depth == 0 && !a.y) : (a.depth >= 1 && (a.weights || a.depth == 1)),
              "%s: either an embedding with ids, or depths with their weights", name);
  PTA_REQUIRE(!a.y || (a.y_weight && pta_aligned(a.y, 16) && pta_aligned(a.y_weight, 16)), "%s: unaligned result, or without its norm's weight", name);
  PTA_REQUIRE(!a.side || (a.table && a.side_table && a.side_layers > 0 && a.side_ld > 0 && a.side_ld % 8 == 0 && pta_aligned(a.side, 16) &&
                          pta_aligned(a.side_table, 16) && a.side_stride % 8 == 0 && a.side_stride >= (size_t)a.rows * a.side_ld),
              "%s: the tokens' own parts (%d layers of %d) do not fit", name, a.side_layers, a.side_ld);
  if (a.router) {
    const int rc = check_routing(a.routing, name);
    if (rc) return rc;
    PTA_REQUIRE(a.h_ld % 8 == 0 && pta_aligned(a.router, 16), "%s: a router reads h, in whole pieces of eight", name);
  }
  hipStream_t s = (hipStream_t)stream;
  const size_t smem = (size_t)a.h_ld * sizeof(float);
  // few rows: a whole row of 1024 threads shortens the chain of a row; many rows: the machine is full either way
  auto launch = [&](auto threads) {
    constexpr int N = decltype(threads)::value;
    if (a.dtype == PTA_BF16) hipLaunchKernelGGL((depth_norm_kernel<bf16, N>), dim3(a.rows), dim3(N), smem, s, a);
    else hipLaunchKernelGGL((depth_norm_kernel<float, N>), dim3(a.rows), dim3(N), smem, s, a);
  };
  if (a.rows <= 64 && a.width >= 2048) launch(std::integral_constant<int, 1024>{});
  else launch(std::integral_constant<int, 256>{});
  PTA_CHECK_LAUNCH(name);
  return PTA_OK;
}

// Eight columns of a row per thread: x += the weighted parts, h = x.
template <typename T>
__global__ __launch_bounds__(256) void add_parts_kernel(pta_add_parts_args a, int pieces) {
  const size_t idx = (size_t)blockIdx.x * 256 + threadIdx.x;
  const size_t r = idx / pieces;
  if (r >= (size_t)a.rows) return;
  const int c = (int)(idx % pieces) * 8, left = a.width - c;
  const bool vec = left >= 8 && (a.width & 7) == 0;
  float* x = a.x + r * a.width + c;
  float v[8];
  load8(x, vec, left, v);
  if (a.parts) {
    const size_t at = r * a.parts_ld * a.width + c;
    const float* w = a.part_weight + r * a.weights_ld;
#pragma unroll 4
    for (int p = 0; p < a.n_parts; ++p) {
      float t[8];
      if (a.part_f32) load8(reinterpret_cast<const float*>(a.parts) + at + (size_t)p * a.width, vec, left, t);
      else load8(reinterpret_cast<const T*>(a.parts) + at + (size_t)p * a.width, vec, left, t);
      const float f = w[p];
#pragma unroll
      for (int e = 0; e < 8; ++e) v[e] = __builtin_fmaf(f, t[e], v[e]);
    }
    if (vec) store8(x, v);
    else for (int e = 0; e < 8 && e < left; ++e) x[e] = v[e];
  }
  store8(reinterpret_cast<T*>(a.h) + r * a.h_ld + c, v);        // (zeros past the width)
}

extern "C" int pta_add_parts(const pta_add_parts_args* args, pta_stream_t stream) {
  const char* name = "pta_add_parts";
  PTA_REQUIRE(args, "%s: null arguments", name);
  const pta_add_parts_args& a = *args;
  PTA_REQUIRE(a.dtype == PTA_BF16 || a.dtype == PTA_FP32, "%s: unknown type %d", name, a.dtype);
  PTA_REQUIRE(a.rows > 0 && a.width > 0 && a.x && a.h && pta_aligned(a.x, 16) && pta_aligned(a.h, 16) && a.h_ld == (a.width + 7) / 8 * 8,
              "%s: rows %d, width %d, h rows of %d", name, a.rows, a.width, a.h_ld);
  PTA_REQUIRE(!a.parts || (a.n_parts >= 1 && a.parts_ld >= a.n_parts && a.part_weight && a.weights_ld >= a.n_parts && pta_aligned(a.parts, 16)),
              "%s: %d parts of %d", name, a.n_parts, a.parts_ld);
  const int pieces = a.h_ld / 8;
  const dim3 grid((unsigned)(((size_t)a.rows * pieces + 255) / 256));
  if (a.dtype == PTA_BF16) hipLaunchKernelGGL((add_parts_kernel<bf16>), grid, dim3(256), 0, (hipStream_t)stream, a, pieces);
  else hipLaunchKernelGGL((add_parts_kernel<float>), grid, dim3(256), 0, (hipStream_t)stream, a, pieces);
  PTA_CHECK_LAUNCH(name);
  return PTA_OK;
}
