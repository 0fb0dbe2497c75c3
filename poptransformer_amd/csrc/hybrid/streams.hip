// Residual streams in fp32, their connections to the sublayers, and the layer norm in front of a sublayer.
#include "hybrid.h"
#include <type_traits>

// One workgroup per row.  A thread owns the columns c, c + 4 * THREADS, ... (four at a time) of every stream, from the
// streams to the normalised result: the row passes through LDS only for the two sums of the norm, and u waits there.
template <typename T, int S, int THREADS>
__global__ __launch_bounds__(THREADS) void streams_norm_kernel(pta_streams_args a, int s_any) {
  constexpr int SMAX = S > 0 ? S : 8;
  constexpr int WAVES = THREADS / 64;
  extern __shared__ __align__(16) float u_row[];
  __shared__ float red[2][WAVES];
  __shared__ float coef[SMAX * SMAX + 2 * SMAX];             // mix | out | in
  const int ns = S > 0 ? S : s_any;
  const int r = blockIdx.x, src = a.gather ? a.gather[r] : r;
  const int d = a.width;
  float* c_mix = coef;
  float* c_out = coef + SMAX * SMAX;
  float* c_in = c_out + SMAX;
  if ((int)threadIdx.x < ns * ns) c_mix[threadIdx.x] = a.y ? a.mix[threadIdx.x] : 0.f;
  if ((int)threadIdx.x < ns) {
    c_out[threadIdx.x] = a.y ? a.mult * a.out[threadIdx.x] : 0.f;
    c_in[threadIdx.x] = a.next_in ? a.next_in[threadIdx.x] : 1.0f;
  }
  const T* row = nullptr;
  if (a.table) {
    int col = a.ids_index ? *a.ids_index : 0;
    col = col < 0 ? 0 : (col >= a.ids_stride ? a.ids_stride - 1 : col);
    int id = a.ids[(size_t)src * a.ids_stride + col];
    id = id < 0 ? 0 : (id >= a.vocab ? a.vocab - 1 : id);
    row = reinterpret_cast<const T*>(a.table) + (size_t)id * d;
    if (a.pos_out && threadIdx.x == 0) a.pos_out[r] = a.ids_index ? *a.ids_index : 0;
  }
  __syncthreads();
  float* xs = a.streams + (size_t)src * ns * d;
  const float* y = a.y ? a.y + (size_t)src * d : nullptr;
  float sum = 0.f;
  auto column = [&](auto width_tag, int c) {
    constexpr int V = decltype(width_tag)::value;
    float x[SMAX][V], u[V] = {}, plain[V] = {};
    auto put = [&](int s, const float (&v)[V]) {
      if (a.write_streams) {
        if constexpr (V == 4) *reinterpret_cast<f32x4*>(xs + (size_t)s * d + c) = f32x4{v[0], v[1], v[2], v[3]};
        else xs[(size_t)s * d + c] = v[0];
      }
#pragma unroll
      for (int e = 0; e < V; ++e) { u[e] = __builtin_fmaf(c_in[s], v[e], u[e]); plain[e] += v[e]; }
    };
    if (row) {
      float v[V];
#pragma unroll
      for (int e = 0; e < V; ++e) v[e] = (float)row[c + e] * a.embed_scale;
#pragma unroll
      for (int s = 0; s < SMAX; ++s)
        if (s < ns) put(s, v);
    } else {
#pragma unroll
      for (int s = 0; s < SMAX; ++s) {
        if (s >= ns) break;
        if constexpr (V == 4) {
          const f32x4 t = *reinterpret_cast<const f32x4*>(xs + (size_t)s * d + c);
#pragma unroll
          for (int e = 0; e < 4; ++e) x[s][e] = t[e];
        } else {
          x[s][0] = xs[(size_t)s * d + c];
        }
      }
      float yv[V] = {};
      if (y) {
        if constexpr (V == 4) {
          const f32x4 t = *reinterpret_cast<const f32x4*>(y + c);
#pragma unroll
          for (int e = 0; e < 4; ++e) yv[e] = t[e];
        } else {
          yv[0] = y[c];
        }
      }
#pragma unroll
      for (int t = 0; t < SMAX; ++t) {
        if (t >= ns) break;
        float v[V];
        if (y) {
#pragma unroll
          for (int e = 0; e < V; ++e) v[e] = c_out[t] * yv[e];
#pragma unroll
          for (int s = 0; s < SMAX; ++s) {
            if (s >= ns) break;
            const float w = c_mix[s * ns + t];
#pragma unroll
            for (int e = 0; e < V; ++e) v[e] = __builtin_fmaf(w, x[s][e], v[e]);
          }
        } else {
#pragma unroll
          for (int e = 0; e < V; ++e) v[e] = x[t][e];
        }
        put(t, v);
      }
    }
#pragma unroll
    for (int e = 0; e < V; ++e) { u_row[c + e] = u[e]; sum += u[e]; }
    if (a.sum_out) {
#pragma unroll
      for (int e = 0; e < V; ++e) a.sum_out[(size_t)r * d + c + e] = plain[e];
    }
  };
  const bool vec = (d & 3) == 0;
  if (vec) for (int c = threadIdx.x * 4; c < d; c += THREADS * 4) column(std::integral_constant<int, 4>{}, c);
  else for (int c = threadIdx.x; c < d; c += THREADS) column(std::integral_constant<int, 1>{}, c);
  if (!a.h) return;
  const float mean = workgroup_sum<WAVES>(sum, red[0]) / (float)d;
  float sq = 0.f;
  const int step = vec ? THREADS * 4 : THREADS, span = vec ? 4 : 1;
  for (int c = threadIdx.x * span; c < d; c += step)
    for (int e = 0; e < span; ++e) { const float t = u_row[c + e] - mean; sq = __builtin_fmaf(t, t, sq); }
  const float var = workgroup_sum<WAVES>(sq, red[1]) / (float)d;
  const float inv = 1.0f / sqrtf(var + a.eps);
  T* h = reinterpret_cast<T*>(a.h) + (size_t)r * a.h_ld;
  for (int c = threadIdx.x * span; c < d; c += step)
    for (int e = 0; e < span; ++e) h[c + e] = (T)((u_row[c + e] - mean) * inv * a.weight[c + e]);
  for (int c = d + threadIdx.x; c < a.h_ld; c += THREADS) h[c] = (T)0.0f;
}

template <typename T, int S>
static int launch_streams(const pta_streams_args& a, hipStream_t s) {
  const size_t smem = (size_t)a.width * sizeof(float);
  // few rows: a whole row of 1024 threads shortens the chain of a row; many rows: the machine is full either way
  if (a.rows <= 64 && a.width >= 2048)
    hipLaunchKernelGGL((streams_norm_kernel<T, S, 1024>), dim3(a.rows), dim3(1024), smem, s, a, a.S);
  else
    hipLaunchKernelGGL((streams_norm_kernel<T, S, 256>), dim3(a.rows), dim3(256), smem, s, a, a.S);
  PTA_CHECK_LAUNCH("pta_streams_norm");
  return PTA_OK;
}

template <typename T>
static int dispatch_streams(const pta_streams_args& a, hipStream_t s) {
  switch (a.S) {
    case 1: return launch_streams<T, 1>(a, s);
    case 2: return launch_streams<T, 2>(a, s);
    case 4: return launch_streams<T, 4>(a, s);
    default: return launch_streams<T, 0>(a, s);
  }
}

extern "C" int pta_streams_norm(const pta_streams_args* args, pta_stream_t stream) {
  PTA_REQUIRE(args, "pta_streams_norm: null arguments");
  const pta_streams_args& a = *args;
  PTA_REQUIRE(a.dtype == PTA_BF16 || a.dtype == PTA_FP32, "pta_streams_norm: unknown type %d", a.dtype);
  PTA_REQUIRE(a.rows > 0 && a.width > 0 && a.width <= 16000, "pta_streams_norm: rows %d, width %d (1 .. 16000)", a.rows, a.width);
  PTA_REQUIRE(a.S >= 1 && a.S <= 8, "pta_streams_norm: 1 to 8 streams, got %d", a.S);
  PTA_REQUIRE(a.streams && pta_aligned(a.streams, 16), "pta_streams_norm: streams null or unaligned");
  PTA_REQUIRE(!a.table || (a.ids && a.vocab > 0 && a.ids_stride > 0 && !a.y), "pta_streams_norm: the embedding needs ids, and no y");
  PTA_REQUIRE(!a.y || (a.out && a.mix && pta_aligned(a.y, 16)), "pta_streams_norm: y needs its connections");
  PTA_REQUIRE(!a.h || (a.weight && a.h_ld >= a.width), "pta_streams_norm: h needs the norm's weight and h_ld >= width");
  PTA_REQUIRE(!a.gather || !a.write_streams, "pta_streams_norm: gathered rows are not written back");
  return a.dtype == PTA_BF16 ? dispatch_streams<bf16>(a, (hipStream_t)stream) : dispatch_streams<float>(a, (hipStream_t)stream);
}
