// State-space recurrence of Mamba-2: token by token (matrix_memory.h has it in chunks on the matrix unit), a row's short convolution
// within the same launch where every sequence has one row; and the gated norm of what it gives.
#include "matrix_memory.h"
#include "short_conv.h"

typedef pta_ssd_args SA;

extern "C" size_t pta_ssd_state_floats(int H, int D, int E) {
  if (H <= 0 || D <= 0 || E <= 0) return 0;
  return (size_t)H * ((E + SL - 1) / SL) * Memory<SA>::slice(D);
}

// ------------------------------------------------------------------------------------------
// A workgroup per (sequence, head, slice of SL value columns) keeps its part of S in registers over the rows of the pass.
// Thread (c4 = tid % 8, y = tid / 8) holds columns 4 c4 .. 4 c4 + 3 of the rows y, y + 32, ... of S.
// CONV: one row per sequence, x, b and c as projected (one behind the other), the convolution's ring brought up to date.
// ------------------------------------------------------------------------------------------
template <typename T, int RPT, bool CONV>
__global__ __launch_bounds__(256) void ssd_scan_kernel(SA a) {
  constexpr int DM = RPT * 32;
  __shared__ __align__(16) float part[2][4][8][4];
  __shared__ __align__(16) float s_b[DM], s_c[DM], s_x[SL];
  const int slices = (a.E + SL - 1) / SL;
  int blk = blockIdx.x;
  const int slice = blk % slices; blk /= slices;
  const int head = blk % a.H, seq = blk / a.H;
  const int c4 = threadIdx.x & 7, y = threadIdx.x >> 3, wave = threadIdx.x >> 6;
  const int D = a.D, E = a.E, per_group = a.H / a.G, group = head / per_group;
  const int row0 = CONV ? seq : a.seq_row[seq], count = CONV ? 1 : a.seq_count[seq], slot = a.slot[row0];
  float* st = a.state + (((size_t)slot * a.H + head) * slices + slice) * Memory<SA>::slice(D);
  f32x4 S[RPT];
#pragma unroll
  for (int k = 0; k < RPT; ++k) {
    const int d = y + 32 * k;
    S[k] = *reinterpret_cast<const f32x4*>(st + (size_t)(d < D ? d : 0) * SL + c4 * 4);
  }
  const float dt_bias = a.dt_bias[head], rate = -expf(a.a_log[head]), direct = a.skip[head];
  const T *xb = reinterpret_cast<const T*>(a.x) + (size_t)head * E, *bb = reinterpret_cast<const T*>(a.b) + (size_t)group * D,
          *cb = reinterpret_cast<const T*>(a.c) + (size_t)group * D;
  if constexpr (CONV) {
    // pieces of eight channels: b, c, the slice's x
    const int pos = a.pos[row0], nd = D / 8, cols = E - slice * SL < SL ? E - slice * SL : SL;
    for (int i = threadIdx.x; i < 2 * nd + cols / 8; i += 256) {
      const bool is_x = i >= 2 * nd, is_c = !is_x && i >= nd;
      const int at = (is_x ? i - 2 * nd : is_c ? i - nd : i) * 8;
      const T* src = (is_x ? xb + slice * SL : is_c ? cb : bb) + (size_t)row0 * a.ld + at;
      const int channel = is_x ? head * E + slice * SL + at : a.H * E + (is_c ? a.G * D : 0) + group * D + at;
      float v[8];
      load8(src, true, 8, v);
      if (is_x || (head % per_group == 0 && slice == 0)) store8(conv_place<T>(a.conv, slot, pos, channel), v);
      conv8<T>(a.conv, slot, pos, channel, v);
      store8((is_x ? s_x : is_c ? s_c : s_b) + at, v);
    }
    __syncthreads();
  }
  for (int t = 0; t < count; ++t) {
    const size_t r = row0 + t;
    const float dt = softplus_f32(a.dt[r * a.H + head] + dt_bias), keep = expf(rate * dt);
    float x[4], bv[RPT], cv[RPT];
    if constexpr (CONV) {
#pragma unroll
      for (int e = 0; e < 4; ++e) x[e] = slice * SL + c4 * 4 + e < E ? s_x[c4 * 4 + e] : 0.f;
    } else {
      const T* px = xb + r * a.ld + slice * SL + c4 * 4;
#pragma unroll
      for (int e = 0; e < 4; ++e) x[e] = slice * SL + c4 * 4 + e < E ? (float)px[e] : 0.f;
    }
#pragma unroll
    for (int k = 0; k < RPT; ++k) {
      const int d = y + 32 * k;
      if constexpr (CONV) {
        bv[k] = d < D ? s_b[d] : 0.f;
        cv[k] = d < D ? s_c[d] : 0.f;
      } else {
        bv[k] = d < D ? (float)bb[r * a.ld + d] : 0.f;
        cv[k] = d < D ? (float)cb[r * a.ld + d] : 0.f;
      }
    }
    f32x4 acc = {0.f, 0.f, 0.f, 0.f};
    float xs[4];
#pragma unroll
    for (int e = 0; e < 4; ++e) xs[e] = x[e] * dt;
#pragma unroll
    for (int k = 0; k < RPT; ++k)
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        S[k][e] = __builtin_fmaf(bv[k], xs[e], keep * S[k][e]);
        acc[e] = __builtin_fmaf(cv[k], S[k][e], acc[e]);
      }
    // over the eight rows of a wave, then over the waves (two buffers in turn: one barrier per token)
#pragma unroll
    for (int o = 8; o < 64; o <<= 1)
#pragma unroll
      for (int e = 0; e < 4; ++e) acc[e] += __shfl_xor(acc[e], o, 64);
    const int p = t & 1;
    if ((threadIdx.x & 63) < 8) *reinterpret_cast<f32x4*>(part[p][wave][c4]) = acc;
    __syncthreads();
    if (threadIdx.x < SL) {
      const int col = threadIdx.x, c = slice * SL + col;
      float s = 0.f;
#pragma unroll
      for (int w = 0; w < 4; ++w) s += part[p][w][col >> 2][col & 3];
      if (c < E) {
        const float own = CONV ? s_x[col] : (float)xb[r * a.ld + c];
        a.y[r * a.H * E + (size_t)head * E + c] = __builtin_fmaf(direct, own, s);
      }
    }
  }
#pragma unroll
  for (int k = 0; k < RPT; ++k) {
    const int d = y + 32 * k;
    if (d < D) *reinterpret_cast<f32x4*>(st + (size_t)d * SL + c4 * 4) = S[k];
  }
}

template <typename T, bool CONV>
static void launch_scan(const SA& a, hipStream_t s) {
  const dim3 grid((unsigned)((size_t)a.seqs * a.H * ((a.E + SL - 1) / SL)));
  if (a.D <= 32) hipLaunchKernelGGL((ssd_scan_kernel<T, 1, CONV>), grid, dim3(256), 0, s, a);
  else if (a.D <= 64) hipLaunchKernelGGL((ssd_scan_kernel<T, 2, CONV>), grid, dim3(256), 0, s, a);
  else if (a.D <= 128) hipLaunchKernelGGL((ssd_scan_kernel<T, 4, CONV>), grid, dim3(256), 0, s, a);
  else if (a.D <= 256) hipLaunchKernelGGL((ssd_scan_kernel<T, 8, CONV>), grid, dim3(256), 0, s, a);
  else hipLaunchKernelGGL((ssd_scan_kernel<T, 16, CONV>), grid, dim3(256), 0, s, a);
}

extern "C" size_t pta_ssd_workspace_bytes(const SA* args) { return chunk_workspace_bytes(args); }

extern "C" int pta_ssd(const SA* args, pta_stream_t stream) {
  const char* name = "pta_ssd";
  PTA_REQUIRE(args, "%s: null arguments", name);
  const SA& a = *args;
  PTA_REQUIRE(a.dtype == PTA_BF16 || a.dtype == PTA_FP32, "%s: unknown type %d", name, a.dtype);
  PTA_REQUIRE(a.rows > 0 && a.seqs > 0 && a.H > 0 && a.G > 0 && a.H % a.G == 0 && a.D > 0 && a.D <= 512 && a.D % 8 == 0 && a.E > 0 && a.E % 8 == 0,
              "%s: rows %d, sequences %d, heads %d in %d groups, sizes %d (multiples of 8 up to 512) and %d (multiples of 8)", name, a.rows, a.seqs,
              a.H, a.G, a.D, a.E);
  PTA_REQUIRE(a.x && a.b && a.c && a.dt && a.dt_bias && a.a_log && a.skip && a.state && a.slot && a.y, "%s: null pointer", name);
  PTA_REQUIRE(pta_aligned(a.x, 16) && pta_aligned(a.b, 16) && pta_aligned(a.c, 16) && pta_aligned(a.state, 16) && pta_aligned(a.y, 16) &&
              a.ld % 8 == 0 && a.ld >= a.H * a.E, "%s: unaligned operand, or rows of %d", name, a.ld);
  hipStream_t s = (hipStream_t)stream;
  if (a.conv.ring) {
    const int rc = check_conv(a.conv, name);
    if (rc) return rc;
    PTA_REQUIRE(a.rows == a.seqs && a.pos && a.conv.channels == a.H * a.E + 2 * a.G * a.D,
                "%s: the convolution takes one row per sequence and %d channels", name, a.H * a.E + 2 * a.G * a.D);
    if (a.dtype == PTA_BF16) launch_scan<bf16, true>(a, s);
    else launch_scan<float, true>(a, s);
  } else {
    PTA_REQUIRE(a.seq_row && a.seq_count && a.longest >= 1 && a.longest <= a.rows, "%s: the sequences' rows are missing (the longest: %d of %d)", name,
                a.longest, a.rows);
    int rc = PTA_OK;
    if (a.dtype == PTA_FP32) launch_scan<float, false>(a, s);
    else if (!a.chunked || a.D > 256) launch_scan<bf16, false>(a, s);
    else if (a.D <= 32) rc = launch_chunk<SA, 1, true>(a, s, name);
    else if (a.D <= 64) rc = launch_chunk<SA, 2, true>(a, s, name);
    else if (a.D <= 128) rc = launch_chunk<SA, 4, true>(a, s, name);
    else rc = launch_chunk<SA, 8, true>(a, s, name);
    if (rc) return rc;
  }
  PTA_CHECK_LAUNCH(name);
  return PTA_OK;
}

// ------------------------------------------------------------------------------------------
// y silu(z), every part over its own root mean square, times the weight: a workgroup per (row, part).  Columns are heads of E of which
// `vdim` count; the parts are equal stretches of the columns that count.
// ------------------------------------------------------------------------------------------
template <typename T, int THREADS>
__global__ __launch_bounds__(THREADS) void gated_norm_kernel(pta_gated_norm_args a) {
  constexpr int WAVES = THREADS / 64, KEEP = 2;               // pieces of eight columns a thread keeps
  __shared__ float red[WAVES];
  const int r = blockIdx.x, part = blockIdx.y, inner = a.H * a.vdim, size = inner / a.parts;
  const int lo = part * size, hi = lo + size;                 // of the columns that count
  const int c_lo = lo / a.vdim * a.E + lo % a.vdim, c_hi = (hi - 1) / a.vdim * a.E + (hi - 1) % a.vdim + 1;
  const float* y = a.y + (size_t)r * a.H * a.E;
  const T* z = reinterpret_cast<const T*>(a.z) + (size_t)r * a.ld_z;
  T* out = reinterpret_cast<T*>(a.out) + (size_t)r * a.H * a.E;
  const int first = c_lo / 8, pieces = (c_hi + 7) / 8 - first;
  const bool whole = c_lo % 8 == 0 && c_hi % 8 == 0;          // no piece holds columns of two parts
  auto gated = [&](int i, float (&v)[8]) {
    float g[8];
    const int c = (first + i) * 8;
    load8(y + c, true, 8, v);
    load8(z + c, true, 8, g);
#pragma unroll
    for (int e = 0; e < 8; ++e) v[e] = whole || (c + e >= c_lo && c + e < c_hi) ? v[e] * silu_of<T>(g[e]) : 0.f;
  };
  float v[KEEP][8], w[KEEP][8], sq = 0.f;
#pragma unroll
  for (int k = 0; k < KEEP; ++k) {
    const int i = threadIdx.x + k * THREADS;
    if (i >= pieces) continue;
    gated(i, v[k]);
    load8(a.weight + (first + i) * 8, true, 8, w[k]);
#pragma unroll
    for (int e = 0; e < 8; ++e) sq = __builtin_fmaf(v[k][e], v[k][e], sq);
  }
  for (int i = threadIdx.x + KEEP * THREADS; i < pieces; i += THREADS) {
    float u[8];
    gated(i, u);
#pragma unroll
    for (int e = 0; e < 8; ++e) sq = __builtin_fmaf(u[e], u[e], sq);
  }
  const float inv = 1.0f / sqrtf(workgroup_sum<WAVES>(sq, red) / (float)size + a.eps);
  auto put = [&](int i, float (&u)[8], const float (&f)[8]) {
    const int c = (first + i) * 8;
#pragma unroll
    for (int e = 0; e < 8; ++e) u[e] = u[e] * inv * f[e];
    if (whole || (c >= c_lo && c + 8 <= c_hi)) {
      store8(out + c, u);
    } else {
      // columns past a head's last belong to the part of that head's last column
      for (int e = 0; e < 8; ++e)
        if (c + e >= c_lo && (c + e < c_hi || (c_hi % a.E == a.vdim && c + e < (c_hi + a.E - 1) / a.E * a.E))) out[c + e] = (T)u[e];
    }
  };
#pragma unroll
  for (int k = 0; k < KEEP; ++k)
    if ((int)threadIdx.x + k * THREADS < pieces) put(threadIdx.x + k * THREADS, v[k], w[k]);
  for (int i = threadIdx.x + KEEP * THREADS; i < pieces; i += THREADS) {
    float u[8], f[8];
    gated(i, u);
    load8(a.weight + (first + i) * 8, true, 8, f);
    put(i, u, f);
  }
}

extern "C" int pta_gated_norm(const pta_gated_norm_args* args, pta_stream_t stream) {
  const char* name = "pta_gated_norm";
  PTA_REQUIRE(args, "%s: null arguments", name);
  const pta_gated_norm_args& a = *args;
  PTA_REQUIRE(a.dtype == PTA_BF16 || a.dtype == PTA_FP32, "%s: unknown type %d", name, a.dtype);
  PTA_REQUIRE(a.rows > 0 && a.H > 0 && a.E > 0 && a.E % 8 == 0 && a.vdim > a.E - 8 && a.vdim <= a.E && a.parts >= 1 && a.parts <= 65535 &&
              a.H * a.vdim % a.parts == 0, "%s: rows %d, %d heads of %d in %d, %d parts", name, a.rows, a.H, a.vdim, a.E, a.parts);
  PTA_REQUIRE(a.y && a.z && a.weight && a.out && pta_aligned(a.y, 16) && pta_aligned(a.z, 16) && pta_aligned(a.weight, 16) && pta_aligned(a.out, 16) &&
              a.ld_z % 8 == 0 && a.ld_z >= a.H * a.E, "%s: null or unaligned operand, gate rows of %d", name, a.ld_z);
  const dim3 grid(a.rows, a.parts);
  const int pieces = a.H * a.E / 8 / a.parts;
  hipStream_t s = (hipStream_t)stream;
  auto launch = [&](auto threads) {
    constexpr int N = decltype(threads)::value;
    if (a.dtype == PTA_BF16) hipLaunchKernelGGL((gated_norm_kernel<bf16, N>), grid, dim3(N), 0, s, a);
    else hipLaunchKernelGGL((gated_norm_kernel<float, N>), grid, dim3(N), 0, s, a);
  };
  if (pieces <= 128) launch(std::integral_constant<int, 64>{});
  else if (pieces <= 512 || a.rows > 64) launch(std::integral_constant<int, 256>{});
  else launch(std::integral_constant<int, 1024>{});
  PTA_CHECK_LAUNCH(name);
  return PTA_OK;
}
