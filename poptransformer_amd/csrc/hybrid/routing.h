// Choice of experts from router logits, shared by the kernels that route rows.
#pragma once
#include "hybrid.h"

// what route_row needs in LDS for a row: logits (then scores), the shared expert's, the groups' scores
constexpr int ROUTE_FLOATS = 2 * PTA_MAX_EXPERTS + 1;
static inline int route_floats(const pta_routing& g) { return g.experts + 1 + g.groups; }

// Routing of row r by THREADS threads, of which this is `tid`: z (route_floats) holds the logits (in LDS, visible to all; overwritten).  Expert e's
// place among the chosen is the number of larger choice scores (of equal ones the first comes first), so no choice waits for another.
// The whole workgroup calls it, each group of THREADS for a row of its own; with `store` unset nothing is kept.  PER: experts of a
// thread, at most (fewer make for less code, whose first fetch is much of a short launch).
template <int THREADS, int PER = (PTA_MAX_EXPERTS + THREADS - 1) / THREADS>
__device__ __forceinline__ void route_row(const pta_routing& g, float* z, int r, int tid, bool store) {
  const int E = g.experts, choices = g.top + g.shared;
  int32_t* chosen = g.chosen + (size_t)r * choices;
  float* weights = g.weights + (size_t)r * choices;
  int rank[PER];
  float p[PER];
  const float shared = g.shared && tid == 0 ? sigmoid_f32(z[E]) : 0.f;
  if (g.score == PTA_SCORE_SIGMOID) {                        // z becomes the choice scores (a thread's own logits only)
#pragma unroll
    for (int k = 0; k < PER; ++k) {
      const int e = tid + k * THREADS;
      p[k] = 0.f;
      if (e >= E) continue;
      p[k] = sigmoid_f32(z[e]);
      z[e] = p[k] + (g.correction ? g.correction[e] : 0.f);
    }
    __syncthreads();
  }
  if (g.keep < g.groups) {                                   // experts of the groups that are not kept leave the choice
    const int size = E / g.groups;
    float* best = z + E + 1;                                 // the sum of each group's two largest choice scores
    for (int n = tid; n < g.groups; n += THREADS) {
      float a = -INFINITY, b = -INFINITY;
#pragma unroll 4
      for (int j = n * size; j < (n + 1) * size; ++j) {
        const float v = z[j];
        b = fmaxf(b, fminf(a, v));
        a = fmaxf(a, v);
      }
      best[n] = size > 1 ? a + b : a;
    }
    __syncthreads();
    for (int e = tid; e < E; e += THREADS) {
      const float own = best[e / size];
      int above = 0;
      for (int j = 0; j < g.groups; ++j) above += best[j] > own || (best[j] == own && j < e / size);
      if (above >= g.keep) z[e] = -INFINITY;
    }
    __syncthreads();
  }
#pragma unroll
  for (int k = 0; k < PER; ++k) {
    const int e = tid + k * THREADS;
    rank[k] = E;
    if (e >= E) continue;
    const float mine = z[e];
    float top = mine;
    int above = 0;
#pragma unroll 8
    for (int j = 0; j < E; ++j) {
      const float v = z[j];
      top = fmaxf(top, v);
      above += v > mine || (v == mine && j < e);
    }
    rank[k] = above;
    if (g.score == PTA_SCORE_SOFTMAX) p[k] = expf(mine - top);
  }
  __syncthreads();
#pragma unroll
  for (int k = 0; k < PER; ++k)                              // what a weight is a share of
    if (tid + k * THREADS < E) z[tid + k * THREADS] = !g.share || rank[k] < g.top ? p[k] : 0.f;
  __syncthreads();
  bool any = false;
#pragma unroll
  for (int k = 0; k < PER; ++k) any = any || rank[k] < g.top;
  if (any && store) {
    float sum = 1.0f;
    if (g.share || g.score == PTA_SCORE_SOFTMAX) {
      sum = g.share ? 1e-20f : 0.f;
#pragma unroll 8
      for (int j = 0; j < E; ++j) sum += z[j];
    }
#pragma unroll
    for (int k = 0; k < PER; ++k)
      if (rank[k] < g.top) {
        chosen[rank[k]] = tid + k * THREADS;
        weights[rank[k]] = p[k] / sum * g.scale;
      }
  }
  if (g.shared && store && tid == 0) {
    chosen[g.top] = E;
    weights[g.top] = shared;
  }
}

// The router's products with a row of `width` values in u (LDS, h_ld of them, the rest is zeroed here), one wave per expert at a time;
// z is visible to all afterwards.
template <typename T, int WAVES>
__device__ __forceinline__ void router_logits(const void* router, int h_ld, int width, float* u, const pta_routing& g, float* z) {
  for (int c = width + threadIdx.x; c < h_ld; c += WAVES * 64) u[c] = 0.f;
  __syncthreads();
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, n = g.experts + g.shared;
  for (int e = wave; e < n; e += WAVES) {
    const T* w = reinterpret_cast<const T*>(router) + (size_t)e * h_ld;
    float s = 0.f;
#pragma unroll 4
    for (int c = lane * 8; c < h_ld; c += 512) {
      float t[8];
      load8(w + c, true, 8, t);
#pragma unroll
      for (int k = 0; k < 8; ++k) s = __builtin_fmaf(t[k], u[c + k], s);
    }
    s = wave_total_dpp(s);
    if (lane == 0) z[e] = s;
  }
  __syncthreads();
}

static inline int check_routing(const pta_routing& g, const char* name) {
  PTA_REQUIRE(g.experts >= 1 && g.experts <= PTA_MAX_EXPERTS && g.top >= 1 && g.top <= g.experts && (g.shared == 0 || g.shared == 1),
              "%s: top %d of %d experts (at most %d)", name, g.top, g.experts, PTA_MAX_EXPERTS);
  PTA_REQUIRE(g.score == PTA_SCORE_SOFTMAX || g.score == PTA_SCORE_SIGMOID, "%s: unknown score %d", name, g.score);
  PTA_REQUIRE(!g.correction || g.score == PTA_SCORE_SIGMOID, "%s: corrections belong to sigmoid scores", name);
  PTA_REQUIRE(g.groups >= 1 && g.experts % g.groups == 0 && g.keep >= 1 && g.keep <= g.groups && g.experts / g.groups * g.keep >= g.top,
              "%s: %d of %d groups of %d experts", name, g.keep, g.groups, g.experts);
  PTA_REQUIRE(g.score == PTA_SCORE_SIGMOID || g.groups == 1, "%s: groups belong to sigmoid scores", name);
  PTA_REQUIRE(g.chosen && g.weights, "%s: the routing has nowhere to go", name);
  return PTA_OK;
}
