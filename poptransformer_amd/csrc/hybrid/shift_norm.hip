// The front of a layer whose sublayers all read the same fp32 residual: embedding (first layer), RMS norm in groups with
// one weight per sublayer, and the token shift of what the mixer reads.
#include "hybrid.h"
#include <type_traits>

typedef pta_shift_norm_args SN;

constexpr int SN_ROWS = 4;               // rows a workgroup walks through at most (and the row before them)

// many rows: fewer of them made twice; not so few workgroups that their walks show
static int rows_of_a_workgroup(const pta_shift_norm_args& a) {
  const int n = a.rows / 512;
  return !a.shift || n < 1 ? 1 : (n > SN_ROWS ? SN_ROWS : n);
}

// A workgroup takes `rows_each` rows one after the other.  A thread owns the same columns of all of them, so the row before
// (normed, fp32) waits for it in LDS; the row before the first comes from the sequence's state, or is made once more.
// The workgroup that holds a sequence's first row of the pass reads its state, and is also the one that writes it: it
// makes the sequence's last row a second time.
template <typename T, int THREADS>
__global__ __launch_bounds__(THREADS) void shift_norm_kernel(SN a, int rows_each) {
  constexpr int WAVES = THREADS / 64;
  extern __shared__ __align__(16) float smem[];
  const int d = a.width, G = a.groups, gsz = d / G;
  const int per = WAVES > G ? WAVES / G : 1, units = G * per;            // waves per group
  float* u = smem;                                                       // [width] the row
  float* before = u + d;                                                 // [width] the normed row before (with a shift)
  float* part = a.shift ? before + d : before;                           // [units]
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const bool vec = (gsz & 3) == 0;
  const int span = vec ? 4 : 1, step = THREADS * span, c_first = threadIdx.x * span;
  const int piece = (gsz + per - 1) / per;

  auto position = [&](int r) {
    int p = a.ids_index ? *a.ids_index : a.pos[r];
    return p < 0 ? 0 : (p >= a.positions ? a.positions - 1 : p);
  };
  // the row into u, the sums of squares of its groups into part
  auto load = [&](int r, bool store) {
    const int src = a.gather ? a.gather[r] : r;
    float* x = a.x + (size_t)src * d;
    if (a.table) {
      const int p = position(src);
      int col = a.ids_index ? *a.ids_index : 0;
      col = col < 0 ? 0 : (col >= a.ids_stride ? a.ids_stride - 1 : col);
      int id = a.ids[(size_t)src * a.ids_stride + col];
      id = id < 0 ? 0 : (id >= a.vocab ? a.vocab - 1 : id);
      const T* e = reinterpret_cast<const T*>(a.table) + (size_t)id * d;
      const T* q = a.pos_table ? reinterpret_cast<const T*>(a.pos_table) + (size_t)p * d : nullptr;
      for (int c = c_first; c < d; c += step)
        for (int k = 0; k < span; ++k) {
          float v = (float)e[c + k] * a.embed_scale;
          if (q) v += (float)q[c + k];
          u[c + k] = v;
          if (store) x[c + k] = v;
        }
    } else if (vec) {
      for (int c = c_first; c < d; c += step) *reinterpret_cast<f32x4*>(u + c) = *reinterpret_cast<const f32x4*>(x + c);
    } else {
      for (int c = c_first; c < d; c += step) u[c] = x[c];
    }
    __syncthreads();
    for (int n = wave; n < units; n += WAVES) {
      const int g = n / per, lo = g * gsz + (n % per) * piece, end = (g + 1) * gsz, hi = lo + piece < end ? lo + piece : end;
      float s = 0.f;
      for (int c = lo + lane; c < hi; c += 64) s = __builtin_fmaf(u[c], u[c], s);
      s = wave_total_dpp(s);
      if (lane == 0) part[n] = s;
    }
    __syncthreads();
  };
  auto inverse = [&](int c) {
    const int g = c / gsz;
    float s = 0.f;
    for (int k = 0; k < per; ++k) s += part[g * per + k];
    return 1.0f / sqrtf(s / (float)gsz + a.eps);
  };

  const int r0 = blockIdx.x * rows_each, r1 = r0 + rows_each < a.rows ? r0 + rows_each : a.rows;
  for (int r = r0; r < r1; ++r) {
    const int last = a.shift ? (a.last ? a.last[r] : r) : -1;            // >= 0: the first row of its sequence
    float* state = last >= 0 ? a.state + (size_t)a.slot[r] * d : nullptr;
    if (state) {
      const bool start = position(r) == 0;
      for (int c = c_first; c < d; c += step)
        for (int k = 0; k < span; ++k) before[c + k] = start ? 0.f : state[c + k];
    } else if (a.shift && r == r0) {
      load(r - 1, false);
      for (int c = c_first; c < d; c += step) {
        const float inv = inverse(c);
        for (int k = 0; k < span; ++k) before[c + k] = u[c + k] * inv * a.w1[c + k];
      }
    }
    load(r, true);
    T* h1 = reinterpret_cast<T*>(a.h1) + (size_t)r * a.h_ld;
    T* h2 = a.h2 ? reinterpret_cast<T*>(a.h2) + (size_t)r * a.h_ld : nullptr;
    T* hm = a.shift ? reinterpret_cast<T*>(a.hm) + (size_t)r * a.h_ld : nullptr;
    auto column = [&](auto tag, int c) {
      constexpr int V = decltype(tag)::value;
      typedef T vecT __attribute__((ext_vector_type(V)));
      vecT o1, o2, om;
      const float inv = inverse(c);
#pragma unroll
      for (int k = 0; k < V; ++k) {
        const float n = u[c + k] * inv, n1 = n * a.w1[c + k];
        o1[k] = (T)n1;
        if (h2) o2[k] = (T)(n * a.w2[c + k]);
        if (hm) {
          om[k] = (T)(n1 + (before[c + k] - n1) * a.shift[c + k]);
          before[c + k] = n1;
          if (last == r) state[c + k] = n1;
        }
      }
      *reinterpret_cast<vecT*>(h1 + c) = o1;
      if (h2) *reinterpret_cast<vecT*>(h2 + c) = o2;
      if (hm) *reinterpret_cast<vecT*>(hm + c) = om;
    };
    if (vec) for (int c = c_first; c < d; c += step) column(std::integral_constant<int, 4>{}, c);
    else for (int c = c_first; c < d; c += step) column(std::integral_constant<int, 1>{}, c);
    for (int c = d + threadIdx.x; c < a.h_ld; c += THREADS) {
      h1[c] = (T)0.0f;
      if (h2) h2[c] = (T)0.0f;
      if (hm) hm[c] = (T)0.0f;
    }
    if (a.pos_out && threadIdx.x == 0) a.pos_out[r] = position(r);
    if (last > r) {
      load(last, false);
      for (int c = c_first; c < d; c += step) {
        const float inv = inverse(c);
        for (int k = 0; k < span; ++k) state[c + k] = u[c + k] * inv * a.w1[c + k];
      }
    }
  }
}

// The same where a wave's 256 columns always lie in one group (group sizes that are multiples of 256): a thread keeps its
// NC * 4 columns of the row, of the row before and of the weights in registers, the next row is on its way while one is
// worked on, and only the groups' sums pass through LDS.
template <typename T, int THREADS, int NC>
__global__ __launch_bounds__(THREADS) void shift_norm_wide_kernel(SN a, int rows_each) {
  constexpr int WAVES = THREADS / 64;
  typedef T vecT __attribute__((ext_vector_type(4)));
  __shared__ float part[2][WAVES * NC];                                  // sums of squares of 256 columns each
  const int d = a.width, gsz = d / a.groups, blocks = gsz / 256;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  f32x4 w1[NC], w2[NC], mix[NC], x[NC], next[NC], before[NC];
  int col[NC];
#pragma unroll
  for (int k = 0; k < NC; ++k) {
    const int c = (k * THREADS + threadIdx.x) * 4;
    col[k] = c < d ? c : -1;                                             // (a whole wave at a time)
  }
  auto vector = [&](const float* p, int k) { return *reinterpret_cast<const f32x4*>(p + (col[k] >= 0 ? col[k] : 0)); };
  auto position = [&](int r) {
    int p = a.ids_index ? *a.ids_index : a.pos[r];
    return p < 0 ? 0 : (p >= a.positions ? a.positions - 1 : p);
  };
  auto load = [&](int r, f32x4 (&v)[NC]) {
    const int src = a.gather ? a.gather[r] : r;
    if (a.table) {
      const int p = position(src);
      int at = a.ids_index ? *a.ids_index : 0;
      at = at < 0 ? 0 : (at >= a.ids_stride ? a.ids_stride - 1 : at);
      int id = a.ids[(size_t)src * a.ids_stride + at];
      id = id < 0 ? 0 : (id >= a.vocab ? a.vocab - 1 : id);
      const T* e = reinterpret_cast<const T*>(a.table) + (size_t)id * d;
      const T* q = reinterpret_cast<const T*>(a.pos_table) + (size_t)p * d;
#pragma unroll
      for (int k = 0; k < NC; ++k) {
        const int c = col[k] >= 0 ? col[k] : 0;
        const vecT ev = *reinterpret_cast<const vecT*>(e + c);
#pragma unroll
        for (int n = 0; n < 4; ++n) v[k][n] = (float)ev[n] * a.embed_scale;
        if (a.pos_table) {
          const vecT qv = *reinterpret_cast<const vecT*>(q + c);
#pragma unroll
          for (int n = 0; n < 4; ++n) v[k][n] += (float)qv[n];
        }
      }
    } else {
#pragma unroll
      for (int k = 0; k < NC; ++k) v[k] = vector(a.x + (size_t)src * d, k);
    }
  };
  int turn = 0;
  float inv[NC];
  auto norms = [&](const f32x4 (&v)[NC]) {                               // inv: of the group of each of the thread's columns
    float* sums = part[turn];
    turn ^= 1;                                                           // (the other half is still being read)
#pragma unroll
    for (int k = 0; k < NC; ++k) {
      float s = 0.f;
#pragma unroll
      for (int n = 0; n < 4; ++n) s = __builtin_fmaf(v[k][n], v[k][n], s);
      s = wave_total_dpp(s);
      if (lane == 0) sums[k * WAVES + wave] = s;                         // block (k * THREADS * 4 + wave * 256) / 256
    }
    __syncthreads();
#pragma unroll
    for (int k = 0; k < NC; ++k) {
      const int g = (col[k] >= 0 ? col[k] : 0) / gsz;
      float s = 0.f;
      for (int b = 0; b < blocks; ++b) s += sums[g * blocks + b];
      inv[k] = 1.0f / sqrtf(s / (float)gsz + a.eps);
    }
  };
  auto normed = [&](const f32x4 (&v)[NC], f32x4 (&out)[NC]) {
    norms(v);
#pragma unroll
    for (int k = 0; k < NC; ++k)
#pragma unroll
      for (int n = 0; n < 4; ++n) out[k][n] = v[k][n] * inv[k] * w1[k][n];
  };

  const int r0 = blockIdx.x * rows_each, r1 = r0 + rows_each < a.rows ? r0 + rows_each : a.rows;
  auto last_of = [&](int r) { return a.shift ? (a.last ? a.last[r] : r) : -1; };
  const bool inside = a.shift && last_of(r0) < 0;                        // the row before r0 is its sequence's
  load(inside ? r0 - 1 : r0, next);
#pragma unroll
  for (int k = 0; k < NC; ++k) {
    w1[k] = vector(a.w1, k);
    if (a.h2) w2[k] = vector(a.w2, k);
    if (a.shift) mix[k] = vector(a.shift, k);
  }
  if (inside) {
#pragma unroll
    for (int k = 0; k < NC; ++k) x[k] = next[k];
    load(r0, next);
    normed(x, before);
  }
  for (int r = r0; r < r1; ++r) {
    const int last = last_of(r);
    float* state = last >= 0 ? a.state + (size_t)a.slot[r] * d : nullptr;
#pragma unroll
    for (int k = 0; k < NC; ++k) x[k] = next[k];
    if (r + 1 < r1) load(r + 1, next);
    if (state) {
      const bool start = position(r) == 0;
#pragma unroll
      for (int k = 0; k < NC; ++k) {
        before[k] = vector(state, k);
#pragma unroll
        for (int n = 0; n < 4; ++n) before[k][n] = start ? 0.f : before[k][n];
      }
    }
    norms(x);
    T* h1 = reinterpret_cast<T*>(a.h1) + (size_t)r * a.h_ld;
    T* h2 = reinterpret_cast<T*>(a.h2) + (size_t)r * a.h_ld;
    T* hm = reinterpret_cast<T*>(a.hm) + (size_t)r * a.h_ld;
#pragma unroll
    for (int k = 0; k < NC; ++k) {
      const int c = col[k];
      if (c < 0) continue;
      vecT o1, o2, om;
      f32x4 n1;
#pragma unroll
      for (int n = 0; n < 4; ++n) {
        const float v = x[k][n] * inv[k];
        n1[n] = v * w1[k][n];
        o1[n] = (T)n1[n];
        if (a.h2) o2[n] = (T)(v * w2[k][n]);
        if (a.shift) om[n] = (T)(n1[n] + (before[k][n] - n1[n]) * mix[k][n]);
      }
      *reinterpret_cast<vecT*>(h1 + c) = o1;
      if (a.h2) *reinterpret_cast<vecT*>(h2 + c) = o2;
      if (a.shift) {
        *reinterpret_cast<vecT*>(hm + c) = om;
        before[k] = n1;
        if (last == r) *reinterpret_cast<f32x4*>(state + c) = n1;
      }
      if (a.table) *reinterpret_cast<f32x4*>(a.x + (size_t)r * d + c) = x[k];
    }
    if (a.pos_out && threadIdx.x == 0) a.pos_out[r] = position(r);
    if (last > r) {                                                      // (uniform: the state of a longer portion)
      f32x4 n1[NC];
      load(last, x);
      normed(x, n1);
#pragma unroll
      for (int k = 0; k < NC; ++k)
        if (col[k] >= 0) *reinterpret_cast<f32x4*>(state + col[k]) = n1[k];
    }
  }
}

template <typename T, int THREADS, int NC>
static void launch_wide(const SN& a, int rows_each, hipStream_t s) {
  hipLaunchKernelGGL((shift_norm_wide_kernel<T, THREADS, NC>), dim3((a.rows + rows_each - 1) / rows_each), dim3(THREADS), 0, s, a, rows_each);
}

template <typename T>
static int launch_shift_norm(const SN& a, hipStream_t s) {
  const bool few = a.rows <= 64 && a.width >= 2048;        // a row of 1024 threads shortens the chain of a row
  const int rows_each = rows_of_a_workgroup(a);
  if ((a.width / a.groups) % 256 == 0 && a.h_ld == a.width) {
    if (few || a.width > 4096) {
      if (a.width <= 4096) launch_wide<T, 1024, 1>(a, rows_each, s);
      else if (a.width <= 8192) launch_wide<T, 1024, 2>(a, rows_each, s);
      else launch_wide<T, 1024, 4>(a, rows_each, s);
    } else if (a.width <= 1024) launch_wide<T, 256, 1>(a, rows_each, s);
    else if (a.width <= 2048) launch_wide<T, 512, 1>(a, rows_each, s);
    else launch_wide<T, 512, 2>(a, rows_each, s);      // (2048 rows of 4096: 22.6 us; with 256 x 4 columns 26.1, 1024 x 1 25.6)
    PTA_CHECK_LAUNCH("pta_shift_norm");
    return PTA_OK;
  }
  const int waves = few ? 16 : 4, per = waves > a.groups ? waves / a.groups : 1;
  const size_t smem = ((size_t)a.width * (a.shift ? 2 : 1) + (size_t)a.groups * per) * sizeof(float);
  const dim3 grid((a.rows + rows_each - 1) / rows_each);
  auto launch = [&](auto tag) -> int {
    constexpr int THREADS = decltype(tag)::value;
    if (smem > 64 * 1024)
      PTA_REQUIRE(hipFuncSetAttribute((const void*)shift_norm_kernel<T, THREADS>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)smem) ==
                  hipSuccess, "pta_shift_norm: %zu bytes of LDS refused", smem);
    hipLaunchKernelGGL((shift_norm_kernel<T, THREADS>), grid, dim3(THREADS), smem, s, a, rows_each);
    return PTA_OK;
  };
  const int rc = few ? launch(std::integral_constant<int, 1024>{}) : launch(std::integral_constant<int, 256>{});
  if (rc) return rc;
  PTA_CHECK_LAUNCH("pta_shift_norm");
  return PTA_OK;
}

extern "C" int pta_shift_norm(const SN* args, pta_stream_t stream) {
  PTA_REQUIRE(args, "pta_shift_norm: null arguments");
  const SN& a = *args;
  PTA_REQUIRE(a.dtype == PTA_BF16 || a.dtype == PTA_FP32, "pta_shift_norm: unknown type %d", a.dtype);
  PTA_REQUIRE(a.rows > 0 && a.width > 0 && a.width <= 16000, "pta_shift_norm: rows %d, width %d (1 .. 16000)", a.rows, a.width);
  PTA_REQUIRE(a.groups > 0 && a.groups <= 1024 && a.width % a.groups == 0, "pta_shift_norm: %d groups of a width of %d", a.groups, a.width);
  PTA_REQUIRE(a.x && a.w1 && a.h1 && a.h_ld >= a.width && pta_aligned(a.x, 16), "pta_shift_norm: null or unaligned operand");
  PTA_REQUIRE(!a.h2 || a.w2, "pta_shift_norm: the second result needs its weight");
  PTA_REQUIRE(!a.shift || (a.hm && a.state && a.slot && (a.pos || a.ids_index) && a.positions > 0),
              "pta_shift_norm: the token shift needs its result, the state, and the rows' slots and positions");
  PTA_REQUIRE(!a.table || (a.ids && a.vocab > 0 && a.ids_stride > 0 && (a.pos || a.ids_index) && a.positions > 0),
              "pta_shift_norm: the embedding needs ids and positions");
  PTA_REQUIRE(!a.gather || (!a.shift && !a.table), "pta_shift_norm: gathered rows take neither a shift nor the embedding");
  PTA_REQUIRE(a.h_ld % 8 == 0 && pta_aligned(a.h1, 16) && (!a.h2 || pta_aligned(a.h2, 16)) && (!a.shift || pta_aligned(a.hm, 16)),
              "pta_shift_norm: results must be 16-byte aligned rows");
  PTA_REQUIRE(pta_aligned(a.w1, 16) && (!a.w2 || pta_aligned(a.w2, 16)) && (!a.shift || (pta_aligned(a.shift, 16) && pta_aligned(a.state, 16))) &&
              (!a.table || pta_aligned(a.table, 16)) && (!a.pos_table || pta_aligned(a.pos_table, 16)), "pta_shift_norm: unaligned operand");
  return a.dtype == PTA_BF16 ? launch_shift_norm<bf16>(a, (hipStream_t)stream) : launch_shift_norm<float>(a, (hipStream_t)stream);
}
