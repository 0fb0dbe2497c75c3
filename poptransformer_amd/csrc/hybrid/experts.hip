// Mixture of experts: every chosen expert's weights are read once, by up to 16 rows directly or by tiles of listed rows.
#include "hybrid.h"
#include "../formats.h"

typedef pta_experts_args EA;

// ------------------------------------------------------------------------------------------
// Lists: which assignments belong to which expert
// ------------------------------------------------------------------------------------------
struct ListLayout {
  int begin, order, tiles, max_tiles, size;
  __host__ __device__ ListLayout(int assignments, int experts, int tile_rows) {
    begin = 4;                                            // [0]: number of tiles
    order = begin + (experts + 1 + 3) / 4 * 4;
    tiles = order + (assignments + 3) / 4 * 4;
    max_tiles = assignments / tile_rows + (experts < assignments ? experts : assignments);
    size = tiles + 4 * max_tiles;
  }
};

__global__ __launch_bounds__(1024) void group_experts_kernel(const int32_t* chosen, int assignments, int top, int choices, int experts,
                                                             int tile_rows, int32_t* lists, ListLayout at) {
  __shared__ int count[1024], first[2][1024], tile[2][1024];
  const int e = threadIdx.x;
  count[e] = 0;
  __syncthreads();
  for (int n = e; n < assignments; n += 1024) {
    const int c = chosen[n / top * choices + n % top];
    if (c >= 0 && c < experts) atomicAdd(&count[c], 1);
  }
  __syncthreads();
  const int mine = count[e], my_tiles = (mine + tile_rows - 1) / tile_rows;
  int cur = 0;
  first[0][e] = mine;
  tile[0][e] = my_tiles;
  __syncthreads();
  for (int d = 1; d < 1024; d <<= 1) {                    // running sums
    first[cur ^ 1][e] = first[cur][e] + (e >= d ? first[cur][e - d] : 0);
    tile[cur ^ 1][e] = tile[cur][e] + (e >= d ? tile[cur][e - d] : 0);
    cur ^= 1;
    __syncthreads();
  }
  const int from = first[cur][e] - mine, tile_from = tile[cur][e] - my_tiles;
  if (e < experts) lists[at.begin + e] = from;
  if (e == experts - 1) {
    lists[at.begin + experts] = from + mine;
    lists[0] = tile_from + my_tiles;
  }
  for (int k = 0; k < my_tiles; ++k) {
    int32_t* t = lists + at.tiles + (tile_from + k) * 4;
    t[0] = e;
    t[1] = from + k * tile_rows;
    t[2] = mine - k * tile_rows < tile_rows ? mine - k * tile_rows : tile_rows;
    t[3] = 0;
  }
  count[e] = from;
  __syncthreads();
  for (int n = e; n < assignments; n += 1024) {
    const int a = n / top * choices + n % top, c = chosen[a];
    if (c >= 0 && c < experts) lists[at.order + atomicAdd(&count[c], 1)] = a;
  }
}

// ------------------------------------------------------------------------------------------
// Directly, up to 16 rows (bf16): a workgroup takes 16 channels (of a pair: of both weights) of one expert that somebody has
// chosen, and finds the rows that have; its waves share the features, their sums meet in LDS.  Workgroups past the experts'
// take the shared expert, which everybody has chosen.
// ------------------------------------------------------------------------------------------
struct DirectMat {
  const unsigned char* W[2];
  size_t expert_bytes;
  int K, KT, blocks, n_main;
  WideOut out;
};

template <bool PAIR, int NW>
__global__ __launch_bounds__(NW * 64) void experts_direct_kernel(EA a, DirectMat routed, DirectMat shared, int slots) {
  constexpr int NACC = PAIR ? 2 : 1;
  __shared__ float red[NW * NACC * 256];
  __shared__ uint32_t present[PTA_MAX_EXPERTS / 32];
  __shared__ int list[16], listed;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const bool is_shared = (int)blockIdx.x >= slots * routed.blocks;
  const DirectMat& mat = is_shared ? shared : routed;
  const int nb = is_shared ? (int)blockIdx.x - slots * routed.blocks : (int)blockIdx.x % routed.blocks;
  const int slot = (int)blockIdx.x / routed.blocks;
  int expert = 0, count;
  if (is_shared) {
    count = a.rows;
    if ((int)threadIdx.x < count) list[threadIdx.x] = threadIdx.x * a.choices + a.top;
    __syncthreads();
  } else if (a.rows == 1) {
    expert = a.chosen[slot];
    count = 1;
    if (threadIdx.x == 0) list[0] = slot;
    __syncthreads();
  } else {
    const int assignments = a.rows * a.top;
    for (int i = threadIdx.x; i < PTA_MAX_EXPERTS / 32; i += NW * 64) present[i] = 0;
    if (threadIdx.x == 0) listed = 0;
    __syncthreads();
    for (int n = threadIdx.x; n < assignments; n += NW * 64) {
      const int e = a.chosen[n / a.top * a.choices + n % a.top];
      if (e >= 0 && e < a.experts) atomicOr(&present[e >> 5], 1u << (e & 31));
    }
    __syncthreads();
    expert = -1;
    int left = slot;
    for (int i = 0; i < (a.experts + 31) / 32; ++i) {     // the expert of this slot: the slot-th of those present
      uint32_t bits = present[i];
      const int here = __popc(bits);
      if (left >= here) { left -= here; continue; }
      for (; left > 0; --left) bits &= bits - 1;
      expert = i * 32 + __ffs(bits) - 1;
      break;
    }
    if (expert < 0) return;                               // fewer experts than slots
    for (int n = threadIdx.x; n < assignments; n += NW * 64) {
      const int at = n / a.top * a.choices + n % a.top;
      if (a.chosen[at] == expert) {
        const int k = atomicAdd(&listed, 1);
        if (k < 16) list[k] = at;
      }
    }
    __syncthreads();
    count = listed < 16 ? listed : 16;
  }
  expert = expert < 0 ? 0 : (expert >= a.experts ? a.experts - 1 : expert);
  const int mine = list[(lane & 15) < count ? (lane & 15) : count - 1];
  const bf16* x = reinterpret_cast<const bf16*>(a.X) + (size_t)(PAIR ? mine / a.choices : mine) * a.ld_x + (lane >> 4) * 8;
  const u32x4* wp[NACC];
#pragma unroll
  for (int g = 0; g < NACC; ++g)
    wp[g] = reinterpret_cast<const u32x4*>(mat.W[g] + (size_t)expert * mat.expert_bytes) + (size_t)nb * mat.KT * 256 + lane;
  f32x4 acc[NACC];
#pragma unroll
  for (int g = 0; g < NACC; ++g) acc[g] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll 2
  for (int kt = wave; kt < mat.KT; kt += NW) {
    u32x4 w[NACC][4];
#pragma unroll
    for (int g = 0; g < NACC; ++g)
#pragma unroll
      for (int v = 0; v < 4; ++v) w[g][v] = __builtin_nontemporal_load(wp[g] + ((size_t)kt * 4 + v) * 64);
    f16x8 xb[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const int k = kt * 128 + j * 32;
      const f16x8 z = {0, 0, 0, 0, 0, 0, 0, 0};
      xb[j] = k + (lane >> 4) * 8 < mat.K ? *reinterpret_cast<const f16x8*>(x + k) : z;
    }
#pragma unroll
    for (int j = 0; j < 4; ++j)
#pragma unroll
      for (int g = 0; g < NACC; ++g) acc[g] = FmtBF16::mma(bitcast<f16x8>(w[g][j]), xb[j], acc[g]);
  }
#pragma unroll
  for (int g = 0; g < NACC; ++g)
#pragma unroll
    for (int r = 0; r < 4; ++r) red[((wave * NACC + g) * 4 + r) * 64 + lane] = acc[g][r];
  __syncthreads();
  for (int idx = threadIdx.x; idx < 256; idx += NW * 64) {
    const int nn = idx & 15, m = idx >> 4, n = nb * 16 + nn;
    if (m >= count || n >= mat.n_main) continue;
    const int r = nn & 3, ln = (nn >> 2) * 16 + m;
    float sum[NACC];
#pragma unroll
    for (int g = 0; g < NACC; ++g) {
      float t = 0.f;
#pragma unroll
      for (int w = 0; w < NW; ++w) t += red[((w * NACC + g) * 4 + r) * 64 + ln];
      sum[g] = t;
    }
    const float y = PAIR ? wide_pair_value(mat.out, n, sum[0], sum[NACC - 1]) : sum[0];
    const size_t at = (size_t)list[m] * a.ld_y + n;
    if (a.out_f32) reinterpret_cast<float*>(a.Y)[at] = y;
    else reinterpret_cast<bf16*>(a.Y)[at] = (bf16)y;
  }
}

// ------------------------------------------------------------------------------------------
// fp32, over the lists: one wave per channel of an expert, eight rows at a time
// ------------------------------------------------------------------------------------------
constexpr int EF_ROWS = 8;

template <bool PAIR>
__global__ __launch_bounds__(256) void experts_f32_kernel(EA a, WideOut out, ListLayout at) {
  const int lane = threadIdx.x & 63, n = blockIdx.x * 4 + (threadIdx.x >> 6), e = blockIdx.y, K = a.routed.K;
  if (n >= a.routed.n_main) return;
  const int begin = a.lists[at.begin + e], end = a.lists[at.begin + e + 1];
  const size_t row = ((size_t)e * a.routed.N + n) * K;
  const float* W = reinterpret_cast<const float*>(a.routed.W) + row;
  const float* W2 = PAIR ? reinterpret_cast<const float*>(a.routed.W2) + row : nullptr;
  for (int b = begin; b < end; b += EF_ROWS) {
    float acc[EF_ROWS] = {}, acc2[EF_ROWS] = {};
    int who[EF_ROWS];
#pragma unroll
    for (int m = 0; m < EF_ROWS; ++m) who[m] = a.lists[at.order + (b + m < end ? b + m : end - 1)];
    for (int k = lane * 4; k < K; k += 256) {
      const f32x4 w = *reinterpret_cast<const f32x4*>(W + k);
      f32x4 w2 = {0.f, 0.f, 0.f, 0.f};
      if (PAIR) w2 = *reinterpret_cast<const f32x4*>(W2 + k);
#pragma unroll
      for (int m = 0; m < EF_ROWS; ++m) {
        const f32x4 x = *reinterpret_cast<const f32x4*>(reinterpret_cast<const float*>(a.X) + (size_t)(PAIR ? who[m] / a.choices : who[m]) * a.ld_x + k);
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          acc[m] = __builtin_fmaf(x[i], w[i], acc[m]);
          if (PAIR) acc2[m] = __builtin_fmaf(x[i], w2[i], acc2[m]);
        }
      }
    }
#pragma unroll
    for (int m = 0; m < EF_ROWS; ++m) {
      const float s = wave_sum(acc[m]), s2 = PAIR ? wave_sum(acc2[m]) : 0.f;
      if (lane == 0 && b + m < end)
        reinterpret_cast<float*>(a.Y)[(size_t)who[m] * a.ld_y + n] = PAIR ? wide_pair_value(out, n, s, s2) : s;
    }
  }
}

// ------------------------------------------------------------------------------------------
static WideOut epilogue_of(const pta_expert_weights& w, const EA& a) {
  WideOut o{};
  o.ld = a.ld_y;
  o.n_main = w.n_main;
  o.out_f32 = a.dtype == PTA_FP32 ? 1 : a.out_f32;
  o.clamped = w.pair == PTA_PAIR_CLAMPED;
  o.limit = w.limit;
  o.slope = w.slope;
  return o;
}

static DirectMat direct_of(const pta_expert_weights& w, const EA& a) {
  DirectMat m{};
  if (!w.W) return m;
  m.W[0] = (const unsigned char*)w.W;
  m.W[1] = (const unsigned char*)w.W2;
  m.expert_bytes = pta_bf16_tiled_bytes(w.N, w.K);
  m.K = w.K;
  m.KT = (w.K + 127) / 128;
  m.blocks = (w.N + 15) / 16;
  m.n_main = w.n_main;
  m.out = epilogue_of(w, a);
  return m;
}

static int check_expert_weights(const pta_expert_weights& w, const EA& a, bool pair, const char* name) {
  PTA_REQUIRE(w.W && pta_aligned(w.W, 16) && (!pair || (w.W2 && pta_aligned(w.W2, 16))), "%s: null or unaligned weights", name);
  PTA_REQUIRE(w.K > 0 && w.K % 8 == 0 && w.K <= a.ld_x && w.n_main >= 1 && w.n_main <= w.N && w.n_main <= a.ld_y,
              "%s: K %d (rows of %d), channels %d of %d (rows of %d)", name, w.K, a.ld_x, w.n_main, w.N, a.ld_y);
  PTA_REQUIRE(a.dtype == PTA_FP32 || w.N % 16 == 0, "%s: %d channels are not whole blocks of 16", name, w.N);
  PTA_REQUIRE(!pair || w.pair == PTA_PAIR_SWIGLU || (w.pair == PTA_PAIR_CLAMPED && w.limit > 0.f), "%s: pair %d, limit %g", name, w.pair, w.limit);
  return PTA_OK;
}

extern "C" size_t pta_expert_lists_size(int rows, int top, int experts, int tile_rows) {
  if (rows <= 0 || top <= 0 || experts <= 0 || tile_rows <= 0) return 0;
  return (size_t)ListLayout(rows * top, experts, tile_rows).size;
}

extern "C" int pta_group_experts(const int32_t* chosen, int rows, int top, int choices, int experts, int tile_rows, int32_t* lists,
                                 pta_stream_t stream) {
  const char* name = "pta_group_experts";
  PTA_REQUIRE(chosen && lists && pta_aligned(lists, 16), "%s: null or unaligned pointer", name);
  PTA_REQUIRE(rows > 0 && rows <= GEMM_MAX_ROWS && top >= 1 && top <= choices && experts >= 1 && experts <= PTA_MAX_EXPERTS &&
              (tile_rows == 128 || tile_rows == 256), "%s: rows %d, top %d of %d experts, tiles of %d", name, rows, top, experts, tile_rows);
  hipLaunchKernelGGL(group_experts_kernel, dim3(1), dim3(1024), 0, (hipStream_t)stream, chosen, rows * top, top, choices, experts, tile_rows,
                     lists, ListLayout(rows * top, experts, tile_rows));
  PTA_CHECK_LAUNCH(name);
  return PTA_OK;
}

template <bool PAIR>
static int launch_direct(const EA& a, hipStream_t s) {
  const DirectMat routed = direct_of(a.routed, a), shared = direct_of(a.shared, a);
  const int all = a.rows * a.top, slots = all < a.experts ? all : a.experts;
  const dim3 grid((unsigned)(slots * routed.blocks + shared.blocks));
  if (routed.KT >= 16) hipLaunchKernelGGL((experts_direct_kernel<PAIR, 8>), grid, dim3(512), 0, s, a, routed, shared, slots);
  else hipLaunchKernelGGL((experts_direct_kernel<PAIR, 4>), grid, dim3(256), 0, s, a, routed, shared, slots);
  return PTA_OK;
}

template <bool PAIR>
static int launch_listed(const EA& a, hipStream_t s, const char* name) {
  const ListLayout at(a.rows * a.top, a.experts, a.tile_rows);
  GemmArgs g{};
  g.count = PAIR ? 2 : 1;
  g.X = (const f16*)a.X;
  g.M = a.rows;
  g.K = a.routed.K;
  g.KT = (g.K + 127) / 128;
  g.mat[0].tiled = a.routed.W;
  g.mat[0].Y = (f16*)a.Y;
  g.mat[0].N = a.routed.N;
  g.mat[0].wide = epilogue_of(a.routed, a);
  if (PAIR) {
    g.mat[1] = g.mat[0];
    g.mat[1].tiled = a.routed.W2;
  }
  make_epilogue(nullptr, &g.epi, name);
  const ListedRows rows{a.lists, a.lists + at.tiles, a.lists + at.order, pta_bf16_tiled_bytes(a.routed.N, a.routed.K), PAIR ? a.choices : 1};
  return a.tile_rows == 256 ? launch_gemm_listed<FmtBF16, 2, PAIR>(g, a.routed.N / 16, at.max_tiles, rows, s, name)
                            : launch_gemm_listed<FmtBF16, 1, PAIR>(g, a.routed.N / 16, at.max_tiles, rows, s, name);
}

extern "C" int pta_experts(const EA* args, pta_stream_t stream) {
  const char* name = "pta_experts";
  PTA_REQUIRE(args, "%s: null arguments", name);
  const EA& a = *args;
  const bool pair = a.routed.W2 != nullptr;
  PTA_REQUIRE(a.dtype == PTA_BF16 || a.dtype == PTA_FP32, "%s: unknown type %d", name, a.dtype);
  PTA_REQUIRE(a.experts >= 1 && a.experts <= PTA_MAX_EXPERTS && a.top >= 1 && a.top <= a.experts && (a.choices == a.top || a.choices == a.top + 1),
              "%s: top %d of %d experts, %d choices", name, a.top, a.experts, a.choices);
  PTA_REQUIRE(a.chosen && a.X && a.Y && pta_aligned(a.X, 16) && pta_aligned(a.Y, 16) && a.ld_x % 8 == 0, "%s: null or unaligned operand", name);
  PTA_REQUIRE(a.rows >= 1 && a.rows <= GEMM_MAX_ROWS, "%s: rows %d (1 .. %d)", name, a.rows, GEMM_MAX_ROWS);
  int rc = check_expert_weights(a.routed, a, pair, name);
  if (!rc && a.shared.W) rc = check_expert_weights(a.shared, a, pair, name);
  if (rc) return rc;
  hipStream_t s = (hipStream_t)stream;
  if (!a.lists) {
    PTA_REQUIRE(a.dtype == PTA_BF16 && a.rows <= 16, "%s: without lists bf16 and up to 16 rows, got %d", name, a.rows);
    PTA_REQUIRE(!a.shared.W || a.choices == a.top + 1, "%s: a shared expert is the last choice", name);
    rc = pair ? launch_direct<true>(a, s) : launch_direct<false>(a, s);
  } else {
    PTA_REQUIRE(!a.shared.W, "%s: the lists do not hold a shared expert", name);
    PTA_REQUIRE((a.tile_rows == 128 || a.tile_rows == 256) && pta_aligned(a.lists, 16), "%s: tiles of %d rows", name, a.tile_rows);
    PTA_REQUIRE(a.dtype == PTA_FP32 || a.ld_x == a.routed.K, "%s: rows of %d, K %d", name, a.ld_x, a.routed.K);
    if (a.dtype == PTA_FP32) {
      const ListLayout at(a.rows * a.top, a.experts, a.tile_rows);
      const dim3 grid((a.routed.n_main + 3) / 4, a.experts);
      if (pair) hipLaunchKernelGGL((experts_f32_kernel<true>), grid, dim3(256), 0, s, a, epilogue_of(a.routed, a), at);
      else hipLaunchKernelGGL((experts_f32_kernel<false>), grid, dim3(256), 0, s, a, epilogue_of(a.routed, a), at);
    } else {
      rc = pair ? launch_listed<true>(a, s, name) : launch_listed<false>(a, s, name);
    }
  }
  if (rc) return rc;
  PTA_CHECK_LAUNCH(name);
  return PTA_OK;
}
