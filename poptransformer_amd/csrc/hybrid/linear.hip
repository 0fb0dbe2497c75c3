// Linear layers with an fp32 epilogue: bf16 operands through the GEMM core, fp32 operands on kernels of their own.
#include "hybrid.h"
#include "../formats.h"

__global__ __launch_bounds__(256) void bf16_tile_kernel(const uint16_t* __restrict__ w, u32x4* __restrict__ tiled, int N, int K,
                                                        int KT, size_t total_vec) {
  const size_t v = (size_t)blockIdx.x * 256 + threadIdx.x;
  if (v >= total_vec) return;
  const int lane = (int)(v & 63), j = (int)((v >> 6) & 3);
  const size_t tile = v >> 8;
  const int kt = (int)(tile % KT), nb = (int)(tile / KT);
  const int row = nb * 16 + (lane & 15), k0 = kt * 128 + j * 32 + (lane >> 4) * 8;
  u32x4 r;
#pragma unroll
  for (int i = 0; i < 4; ++i) {
    const int k = k0 + 2 * i;
    const uint32_t lo = (row < N && k < K) ? w[(size_t)row * K + k] : 0;
    const uint32_t hi = (row < N && k + 1 < K) ? w[(size_t)row * K + k + 1] : 0;
    r[i] = lo | (hi << 16);
  }
  tiled[v] = r;
}

extern "C" size_t pta_bf16_tiled_bytes(int N, int K) { return gemv_tiled_bytes(N, K, FmtBF16::kVec); }

extern "C" int pta_bf16_tile(const uint16_t* w, void* tiled, int N, int K, pta_stream_t stream) {
  PTA_REQUIRE(w && tiled, "pta_bf16_tile: null pointer");
  PTA_REQUIRE(N > 0 && K > 0, "pta_bf16_tile: need N > 0 and K > 0, got N=%d K=%d", N, K);
  PTA_REQUIRE(pta_aligned(tiled, 16), "pta_bf16_tile: tiled buffer must be 16-byte aligned");
  const size_t total = pta_bf16_tiled_bytes(N, K) / 16;
  hipLaunchKernelGGL(bf16_tile_kernel, dim3((unsigned)((total + 255) / 256)), dim3(256), 0, (hipStream_t)stream, w,
                     (u32x4*)tiled, N, K, (K + 127) / 128, total);
  PTA_CHECK_LAUNCH("pta_bf16_tile");
  return PTA_OK;
}

// ------------------------------------------------------------------------------------------
// fp32: up to F32_ROWS rows, one wave per output channel (the channel's weights are read once)
// ------------------------------------------------------------------------------------------
constexpr int F32_ROWS = 8;

template <bool PAIR>
__global__ __launch_bounds__(256) void f32_gemv_kernel(const float* __restrict__ X, const float* __restrict__ W,
                                                       const float* __restrict__ W2, int M, int K, int N, GemmMat mat) {
  const int lane = threadIdx.x & 63;
  const int n = blockIdx.x * 4 + (threadIdx.x >> 6);
  if (n >= N) return;
  float acc[F32_ROWS] = {}, acc2[F32_ROWS] = {};
  for (int k = lane * 4; k < K; k += 256) {
    const f32x4 w = *reinterpret_cast<const f32x4*>(W + (size_t)n * K + k);
    f32x4 w2 = {0.f, 0.f, 0.f, 0.f};
    if (PAIR) w2 = *reinterpret_cast<const f32x4*>(W2 + (size_t)n * K + k);
#pragma unroll
    for (int m = 0; m < F32_ROWS; ++m) {
      if (m >= M) break;
      const f32x4 x = *reinterpret_cast<const f32x4*>(X + (size_t)m * K + k);
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        acc[m] = __builtin_fmaf(x[e], w[e], acc[m]);
        if (PAIR) acc2[m] = __builtin_fmaf(x[e], w2[e], acc2[m]);
      }
    }
  }
#pragma unroll
  for (int m = 0; m < F32_ROWS; ++m) {
    const float s = wave_sum(acc[m]);
    const float s2 = PAIR ? wave_sum(acc2[m]) : 0.f;
    if (lane == 0 && m < M) {
      if (PAIR) wide_put_pair(mat, m, n, s, s2);
      else wide_put(mat, m, n, s);
    }
  }
}

// many rows: 64 x 64 outputs per workgroup, 4 x 4 per thread, 16 features at a time through LDS
template <bool PAIR>
__global__ __launch_bounds__(256) void f32_gemm_kernel(const float* __restrict__ X, const float* __restrict__ W,
                                                       const float* __restrict__ W2, int M, int K, int N, GemmMat mat) {
  constexpr int T = 64, KS = 16, NW = PAIR ? 2 : 1;
  __shared__ float xs[KS][T + 4], ws[NW][KS][T + 4];
  const int tx = threadIdx.x & 15, ty = threadIdx.x >> 4;
  const int m0 = blockIdx.y * T, n0 = blockIdx.x * T;
  const int lr = threadIdx.x >> 2, lk = (threadIdx.x & 3) * 4;      // this thread's four features of one row of a tile
  float acc[NW][4][4] = {};
  for (int k0 = 0; k0 < K; k0 += KS) {
    const int k = k0 + lk;
    const f32x4 z = {0.f, 0.f, 0.f, 0.f};
    const f32x4 xv = (m0 + lr < M && k < K) ? *reinterpret_cast<const f32x4*>(X + (size_t)(m0 + lr) * K + k) : z;
    f32x4 wv[NW];
#pragma unroll
    for (int g = 0; g < NW; ++g)
      wv[g] = (n0 + lr < N && k < K) ? *reinterpret_cast<const f32x4*>((g ? W2 : W) + (size_t)(n0 + lr) * K + k) : z;
    __syncthreads();
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      xs[lk + e][lr] = xv[e];
#pragma unroll
      for (int g = 0; g < NW; ++g) ws[g][lk + e][lr] = wv[g][e];
    }
    __syncthreads();
#pragma unroll
    for (int kk = 0; kk < KS; ++kk) {
      const f32x4 a = *reinterpret_cast<const f32x4*>(&xs[kk][ty * 4]);
#pragma unroll
      for (int g = 0; g < NW; ++g) {
        const f32x4 b = *reinterpret_cast<const f32x4*>(&ws[g][kk][tx * 4]);
#pragma unroll
        for (int i = 0; i < 4; ++i)
#pragma unroll
          for (int j = 0; j < 4; ++j) acc[g][i][j] = __builtin_fmaf(a[i], b[j], acc[g][i][j]);
      }
    }
  }
#pragma unroll
  for (int i = 0; i < 4; ++i)
#pragma unroll
    for (int j = 0; j < 4; ++j) {
      const int m = m0 + ty * 4 + i, n = n0 + tx * 4 + j;
      if (m >= M || n >= N) continue;
      if (PAIR) wide_put_pair(mat, m, n, acc[0][i][j], acc[NW - 1][i][j]);
      else wide_put(mat, m, n, acc[0][i][j]);
    }
}

template <bool PAIR>
static void launch_f32(const pta_wide_linear_args& a, const GemmMat& mat, hipStream_t s) {
  const float *X = (const float*)a.X, *W = (const float*)a.W, *W2 = (const float*)a.W2;
  if (a.M <= F32_ROWS)
    hipLaunchKernelGGL((f32_gemv_kernel<PAIR>), dim3((a.N + 3) / 4), dim3(256), 0, s, X, W, W2, a.M, a.K, a.N, mat);
  else
    hipLaunchKernelGGL((f32_gemm_kernel<PAIR>), dim3((a.N + 63) / 64, (a.M + 63) / 64), dim3(256), 0, s, X, W, W2, a.M, a.K,
                       a.N, mat);
}

extern "C" size_t pta_wide_linear_workspace_bytes(int M, int N) {
  if (M <= 0 || N <= 0) return 0;
  return (size_t)GEMM_MAX_KSPLIT * M * N * sizeof(float);
}

static int check_wide(const pta_wide_linear_args& a, const char* name) {
  const bool pair = a.pair != PTA_PAIR_NONE;
  PTA_REQUIRE(a.dtype == PTA_BF16 || a.dtype == PTA_FP32, "%s: unknown type %d", name, a.dtype);
  PTA_REQUIRE(a.pair >= PTA_PAIR_NONE && a.pair <= PTA_PAIR_CLAMPED, "%s: unknown pair %d", name, a.pair);
  const int rc = check_gemv_common(name, a.X, a.M, a.K);
  if (rc) return rc;
  PTA_REQUIRE(a.W && a.Y && a.N > 0 && pta_aligned(a.W, 16) && pta_aligned(a.Y, 16), "%s: null or unaligned operand", name);
  PTA_REQUIRE(!pair || (a.W2 && pta_aligned(a.W2, 16)), "%s: a pair needs its second weight", name);
  PTA_REQUIRE(a.n_main >= 1 && a.n_main <= a.ld && a.tail_count >= 0 && a.n_main + a.tail_count <= a.N,
              "%s: n_main %d (ld %d) and tail %d do not fit %d channels", name, a.n_main, a.ld, a.tail_count, a.N);
  PTA_REQUIRE(a.tail_count == 0 || (a.tail && !pair), "%s: a tail needs its buffer, and a single weight", name);
  PTA_REQUIRE(a.pair != PTA_PAIR_CLAMPED || a.limit > 0.f, "%s: the clamped pair needs a positive limit", name);
  PTA_REQUIRE(a.act >= PTA_ACT_NONE && a.act <= PTA_ACT_SIGMOID, "%s: unknown activation %d", name, a.act);
  PTA_REQUIRE(pair || !a.bias2, "%s: a second bias belongs to a pair", name);
  PTA_REQUIRE(!a.accumulate || a.out_f32 || a.dtype == PTA_FP32, "%s: only fp32 results accumulate", name);
  PTA_REQUIRE(!a.mul || pta_aligned(a.mul, 16), "%s: the multiplier must be 16-byte aligned", name);
  PTA_REQUIRE(!a.workspace || pta_aligned(a.workspace, 16), "%s: the workspace must be 16-byte aligned", name);
  return PTA_OK;
}

static GemmMat wide_matrix(const pta_wide_linear_args& a, const void* W) {
  GemmMat mat{};
  mat.tiled = W;
  mat.act = PTA_ACT_NONE;
  mat.Y = (f16*)a.Y;
  mat.N = a.N;
  WideOut& w = mat.wide;
  w.ld = a.ld;
  w.n_main = a.n_main;
  w.out_f32 = a.dtype == PTA_FP32 ? 1 : a.out_f32;
  w.tail = a.tail;
  w.tail_count = a.tail_count;
  w.tail_bias = a.tail_bias;
  w.cap = a.cap;
  w.clamped = a.pair == PTA_PAIR_CLAMPED;
  w.limit = a.limit;
  w.slope = a.slope;
  w.bias = a.bias;
  w.bias2 = a.bias2;
  w.act = a.act;
  w.mul = a.mul;
  w.mul_f32 = a.dtype == PTA_FP32;
  w.accumulate = a.accumulate;
  return mat;
}

static int wide_linear(const pta_wide_linear_args& a, hipStream_t s, const char* name) {
  const bool pair = a.pair != PTA_PAIR_NONE;
  if (a.dtype == PTA_FP32) {
    const GemmMat mat = wide_matrix(a, a.W);
    if (pair) launch_f32<true>(a, mat, s);
    else launch_f32<false>(a, mat, s);
    PTA_CHECK_LAUNCH(name);
    return PTA_OK;
  }
  GemmArgs g{};
  g.count = pair ? 2 : 1;
  g.X = (const f16*)a.X;
  g.M = a.M;
  g.K = a.K;
  g.KT = (a.K + 127) / 128;
  g.mat[0] = wide_matrix(a, a.W);
  if (pair) g.mat[1] = wide_matrix(a, a.W2);
  make_epilogue(nullptr, &g.epi, name);
  g.part = (float*)a.workspace;
  g.part_bytes = a.workspace ? a.workspace_bytes : 0;
  const int nb = (a.N + 15) / 16;
  return pair ? dispatch_gemv<FmtBF16, true>(g, nb, s, name) : dispatch_gemv<FmtBF16, false>(g, nb, s, name);
}

extern "C" int pta_wide_linear(const pta_wide_linear_args* args, pta_stream_t stream) {
  PTA_REQUIRE(args, "pta_wide_linear: null arguments");
  const int rc = check_wide(*args, "pta_wide_linear");
  return rc ? rc : wide_linear(*args, (hipStream_t)stream, "pta_wide_linear");
}

extern "C" int pta_wide_linear_group(const pta_wide_linear_args* list, int count, pta_stream_t stream) {
  const char* name = "pta_wide_linear_group";
  PTA_REQUIRE(list && count >= 1 && count <= 4, "%s: 1 to 4 matrices, got %d", name, count);
  for (int i = 0; i < count; ++i) {
    const int rc = check_wide(list[i], name);
    if (rc) return rc;
    PTA_REQUIRE(list[i].pair == PTA_PAIR_NONE && list[i].dtype == list[0].dtype && list[i].M == list[0].M && list[i].K == list[0].K,
                "%s: single matrices with the same rows and features", name);
  }
  hipStream_t s = (hipStream_t)stream;
  // one launch: up to 16 rows, and whole tiles of more than 64 (whose workgroups would not fill the machine evenly one by one)
  bool together = list[0].dtype == PTA_BF16 && (list[0].M <= 16 || (list[0].M > 64 && list[0].K >= 512));
  for (int i = 0; i < count && list[0].M > 64; ++i) together = together && list[i].N % 128 == 0;
  if (!together) {
    for (int i = 0; i < count; ++i) {
      const int rc = wide_linear(list[i], s, name);
      if (rc) return rc;
    }
    return PTA_OK;
  }
  GemmArgs g{};
  g.count = count;
  g.X = (const f16*)list[0].X;
  g.M = list[0].M;
  g.K = list[0].K;
  g.KT = (g.K + 127) / 128;
  int nb = 0;
  for (int i = 0; i < count; ++i) {
    g.mat[i] = wide_matrix(list[i], list[i].W);
    g.mat[i].X = list[i].X != list[0].X ? (const f16*)list[i].X : nullptr;
    g.mat[i].nb_begin = nb;
    nb += (list[i].N + 15) / 16;
  }
  make_epilogue(nullptr, &g.epi, name);
  return dispatch_gemv<FmtBF16, false>(g, nb, s, name);
}
