// Matrix memory (mLSTM): the recurrence token by token (matrix_memory.h has it in chunks on the matrix unit), and the per-head
// norm with the output gate.
#include "matrix_memory.h"

typedef pta_mlstm_args MA;

extern "C" size_t pta_mlstm_state_floats(int H, int D, int E) {
  if (H <= 0 || D <= 0 || E <= 0) return 0;
  const size_t slice = ((size_t)D * SL + D + 2 + 3) / 4 * 4;             // slices start on 16-byte boundaries
  return (size_t)H * ((E + SL - 1) / SL) * slice;
}

// ------------------------------------------------------------------------------------------
// Token by token: a workgroup per (sequence, head, slice of SL value columns) keeps its part of S in registers over the
// rows of the pass (one row in a decode step: the state is read, updated, multiplied and written in one go).  Thread
// (x = tid % 8, y = tid / 8) holds columns 4 x .. 4 x + 3 of the rows y, y + 32, ... of S, and n of those rows.
// ------------------------------------------------------------------------------------------
template <typename T, int RPT>
__global__ __launch_bounds__(256) void mlstm_scan_kernel(MA a) {
  __shared__ __align__(16) float part[2][4][8][4];
  __shared__ float part_n[2][4];
  const int slices = (a.E + SL - 1) / SL;
  int b = blockIdx.x;
  const int slice = b % slices; b /= slices;
  const int head = b % a.H, seq = b / a.H;
  const int x = threadIdx.x & 7, y = threadIdx.x >> 3, wave = threadIdx.x >> 6;
  const bool single = a.rows == a.seqs;                  // one row per sequence: row = sequence
  const int D = a.D, row0 = single ? seq : a.seq_row[seq], count = single ? 1 : a.seq_count[seq];
  const size_t per = Memory<MA>::slice(D);
  float* st = a.state + (((size_t)a.slot[row0] * a.H + head) * slices + slice) * per;
  float *st_n = st + (size_t)D * SL, *st_m = st_n + D;
  f32x4 S[RPT];
  float n[RPT];
#pragma unroll
  for (int k = 0; k < RPT; ++k) {
    const int d = y + 32 * k;
    S[k] = d < D ? *reinterpret_cast<const f32x4*>(st + (size_t)d * SL + x * 4) : f32x4{0.f, 0.f, 0.f, 0.f};
    n[k] = d < D ? st_n[d] : 0.f;
  }
  float m = *st_m;
  const int col = slice * SL + x * 4;                    // first of this thread's value columns of the head
  const float qscale = 1.0f / sqrtf((float)D);
  for (int t = 0; t < count; ++t) {
    const size_t r = row0 + t;
    const T* q = reinterpret_cast<const T*>(a.q) + r * a.ld + (size_t)head * D;
    const T* k_ = reinterpret_cast<const T*>(a.k) + r * a.ld + (size_t)head * D;
    const T* v_ = reinterpret_cast<const T*>(a.v) + r * a.ld + (size_t)head * a.E;
    const float i = log_input_gate(a.gates[r * 2 * a.H + head], a.cap);
    const float f = log_forget_gate(a.gates[r * 2 * a.H + a.H + head], a.cap);
    const float mn = fmaxf(f + m, i), keep = expf(f + m - mn), take = expf(i - mn);
    m = mn;
    float v[4], qv[RPT], kv[RPT];
#pragma unroll
    for (int e = 0; e < 4; ++e) v[e] = col + e < a.E ? (float)v_[col + e] * take : 0.f;
#pragma unroll
    for (int k = 0; k < RPT; ++k) {
      const int d = y + 32 * k;
      qv[k] = d < D ? (float)q[d] * qscale : 0.f;
      kv[k] = d < D ? (float)k_[d] : 0.f;
    }
    f32x4 acc = {0.f, 0.f, 0.f, 0.f};
    float nq = 0.f;
#pragma unroll
    for (int k = 0; k < RPT; ++k) {
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        S[k][e] = __builtin_fmaf(kv[k], v[e], keep * S[k][e]);
        acc[e] = __builtin_fmaf(qv[k], S[k][e], acc[e]);
      }
      n[k] = __builtin_fmaf(take, kv[k], keep * n[k]);
      nq = __builtin_fmaf(qv[k], n[k], nq);
    }
    // over the eight rows of a wave, then over the waves (two buffers in turn: one barrier per token)
#pragma unroll
    for (int o = 8; o < 64; o <<= 1) {
#pragma unroll
      for (int e = 0; e < 4; ++e) acc[e] += __shfl_xor(acc[e], o, 64);
      nq += __shfl_xor(nq, o, 64);
    }
    const int p = t & 1;
    if ((threadIdx.x & 63) < 8) *reinterpret_cast<f32x4*>(part[p][wave][x]) = acc;
    if ((threadIdx.x & 63) == 0) part_n[p][wave] = nq;
    __syncthreads();
    if (threadIdx.x < SL) {
      const int c = slice * SL + threadIdx.x;
      float s = 0.f, d = 0.f;
#pragma unroll
      for (int w = 0; w < 4; ++w) { s += part[p][w][threadIdx.x >> 2][threadIdx.x & 3]; d += part_n[p][w]; }
      if (c < a.E) a.o[r * a.H * a.E + (size_t)head * a.E + c] = s / (fmaxf(fabsf(d), expf(-m)) + 1e-6f);
    }
  }
#pragma unroll
  for (int k = 0; k < RPT; ++k) {
    const int d = y + 32 * k;
    if (d >= D) continue;
    *reinterpret_cast<f32x4*>(st + (size_t)d * SL + x * 4) = S[k];
    if (x == 0) st_n[d] = n[k];
  }
  if (threadIdx.x == 0) *st_m = m;
}

extern "C" size_t pta_mlstm_workspace_bytes(const MA* args) { return chunk_workspace_bytes(args); }

template <int DT>
static int launch_chunks(const MA& a, bool vec, hipStream_t s) {
  return vec ? launch_chunk<MA, DT, true>(a, s, "pta_mlstm") : launch_chunk<MA, DT, false>(a, s, "pta_mlstm");
}

template <typename T>
static void launch_scan(const MA& a, hipStream_t s) {
  const dim3 grid(a.seqs * a.H * ((a.E + SL - 1) / SL));
  if (a.D <= 32) hipLaunchKernelGGL((mlstm_scan_kernel<T, 1>), grid, dim3(256), 0, s, a);
  else if (a.D <= 64) hipLaunchKernelGGL((mlstm_scan_kernel<T, 2>), grid, dim3(256), 0, s, a);
  else if (a.D <= 128) hipLaunchKernelGGL((mlstm_scan_kernel<T, 4>), grid, dim3(256), 0, s, a);
  else if (a.D <= 256) hipLaunchKernelGGL((mlstm_scan_kernel<T, 8>), grid, dim3(256), 0, s, a);
  else hipLaunchKernelGGL((mlstm_scan_kernel<T, 16>), grid, dim3(256), 0, s, a);
}

extern "C" int pta_mlstm(const MA* args, pta_stream_t stream) {
  PTA_REQUIRE(args, "pta_mlstm: null arguments");
  const MA& a = *args;
  PTA_REQUIRE(a.dtype == PTA_BF16 || a.dtype == PTA_FP32, "pta_mlstm: unknown type %d", a.dtype);
  PTA_REQUIRE(a.rows > 0 && a.seqs > 0 && a.H > 0 && a.D > 0 && a.D <= 512 && a.E > 0, "pta_mlstm: rows %d, sequences %d, heads %d, sizes %d (1 .. 512) and %d",
              a.rows, a.seqs, a.H, a.D, a.E);
  PTA_REQUIRE(a.q && a.k && a.v && a.gates && a.state && a.slot && a.seq_row && a.seq_count && a.o, "pta_mlstm: null pointer");
  PTA_REQUIRE(pta_aligned(a.state, 16) && pta_aligned(a.o, 16), "pta_mlstm: state and output must be 16-byte aligned");
  PTA_REQUIRE(a.cap > 0.f && a.ld >= a.H * a.D && a.ld >= a.H * a.E, "pta_mlstm: gate cap %g, row stride %d", (double)a.cap, a.ld);
  hipStream_t s = (hipStream_t)stream;
  if (a.dtype == PTA_FP32) {
    launch_scan<float>(a, s);
  } else if (a.chunked && a.D <= 256) {
    PTA_REQUIRE(a.longest >= 1 && a.longest <= a.rows, "pta_mlstm: longest sequence %d of %d rows", a.longest, a.rows);
    const bool vec = a.D % 8 == 0 && a.E % 8 == 0 && a.ld % 8 == 0 && pta_aligned(a.q, 16) && pta_aligned(a.k, 16) && pta_aligned(a.v, 16);
    int rc;
    if (a.D <= 32) rc = launch_chunks<1>(a, vec, s);
    else if (a.D <= 64) rc = launch_chunks<2>(a, vec, s);
    else if (a.D <= 128) rc = launch_chunks<4>(a, vec, s);
    else rc = launch_chunks<8>(a, vec, s);
    if (rc) return rc;
  } else {
    launch_scan<bf16>(a, s);
  }
  PTA_CHECK_LAUNCH("pta_mlstm");
  return PTA_OK;
}

// ------------------------------------------------------------------------------------------
// Each head's output over its root mean square, times the weight, times sigmoid(gate): one wave per (row, head).
// ------------------------------------------------------------------------------------------
template <typename T>
__global__ __launch_bounds__(256) void head_norm_gate_kernel(const float* __restrict__ o, const float* __restrict__ weight,
                                                             const T* __restrict__ gate, int gate_ld, T* __restrict__ out,
                                                             int out_ld, int rows, int H, int E, float eps, bool vec) {
  constexpr int KEEP = 2;                                    // 8-element pieces of a head a lane keeps in registers
  const int lane = threadIdx.x & 63;
  const int idx = blockIdx.x * 4 + (threadIdx.x >> 6);
  if (idx >= rows * H) return;
  const int r = idx / H, head = idx % H;
  const float* x = o + (size_t)idx * E;
  const T* g = gate + (size_t)r * gate_ld + (size_t)head * E;
  const float* w = weight + (size_t)head * E;
  T* y = out + (size_t)r * out_ld + (size_t)head * E;
  float sq = 0.f;
  if (vec && E <= KEEP * 512) {
    float xv[KEEP][8], gv[KEEP][8], wv[KEEP][8];
#pragma unroll
    for (int k = 0; k < KEEP; ++k) {
      const int e = (k * 64 + lane) * 8, left = E - e;
      load8(x + (left > 0 ? e : 0), left > 0, 0, xv[k]);
      load8(g + (left > 0 ? e : 0), left > 0, 0, gv[k]);
      load8(w + (left > 0 ? e : 0), left > 0, 0, wv[k]);
#pragma unroll
      for (int c = 0; c < 8; ++c) sq = __builtin_fmaf(xv[k][c], xv[k][c], sq);
    }
    const float inv = 1.0f / sqrtf(wave_total_dpp(sq) / (float)E + eps);
#pragma unroll
    for (int k = 0; k < KEEP; ++k) {
      const int e = (k * 64 + lane) * 8;
      if (e >= E) break;
#pragma unroll
      for (int c = 0; c < 8; ++c) xv[k][c] = xv[k][c] * inv * wv[k][c] * sigmoid_f32(gv[k][c]);
      store8(y + e, xv[k]);
    }
  } else {
    for (int e = lane; e < E; e += 64) sq = __builtin_fmaf(x[e], x[e], sq);
    const float inv = 1.0f / sqrtf(wave_total_dpp(sq) / (float)E + eps);
    for (int e = lane; e < E; e += 64) y[e] = (T)(x[e] * inv * w[e] * sigmoid_f32((float)g[e]));
  }
  if (head == 0)
    for (int c = H * E + lane; c < out_ld; c += 64) out[(size_t)r * out_ld + c] = (T)0.0f;
}

extern "C" int pta_head_norm_gate(int dtype, const float* o, const float* weight, const void* gate, int gate_ld, void* out, int out_ld,
                                  int rows, int H, int E, float eps, pta_stream_t stream) {
  PTA_REQUIRE(dtype == PTA_BF16 || dtype == PTA_FP32, "pta_head_norm_gate: unknown type %d", dtype);
  PTA_REQUIRE(o && weight && gate && out, "pta_head_norm_gate: null pointer");
  PTA_REQUIRE(rows > 0 && H > 0 && E > 0 && gate_ld >= H * E && out_ld >= H * E, "pta_head_norm_gate: rows %d, heads %d, size %d, strides %d and %d",
              rows, H, E, gate_ld, out_ld);
  const dim3 grid((rows * H + 3) / 4);
  const int es = dtype == PTA_BF16 ? 2 : 4;
  const bool vec = E % 8 == 0 && (gate_ld * es) % 16 == 0 && (out_ld * es) % 16 == 0 && pta_aligned(o, 16) && pta_aligned(weight, 16) &&
                   pta_aligned(gate, 16) && pta_aligned(out, 16);
  if (dtype == PTA_BF16)
    hipLaunchKernelGGL((head_norm_gate_kernel<bf16>), grid, dim3(256), 0, (hipStream_t)stream, o, weight, (const bf16*)gate, gate_ld,
                       (bf16*)out, out_ld, rows, H, E, eps, vec);
  else
    hipLaunchKernelGGL((head_norm_gate_kernel<float>), grid, dim3(256), 0, (hipStream_t)stream, o, weight, (const float*)gate, gate_ld,
                       (float*)out, out_ld, rows, H, E, eps, vec);
  PTA_CHECK_LAUNCH("pta_head_norm_gate");
  return PTA_OK;
}
