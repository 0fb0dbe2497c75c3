// Attention whose cache holds one latent and one shared rotated key part per token.
//
// Absorbed form: W_uk^T q meets the cached rows, so all heads of a row share every key that is read; the 16 columns of a
// matrix instruction are 16 heads.  Over heads: prompts, with keys and values of every head in buffers of their own.
#include "attention.h"

typedef pta_latent_args LA;

__device__ __forceinline__ int position_of(const LA& a, int r) {
  const int p = a.pos[r];
  return p < 0 ? 0 : (p >= a.positions ? a.positions - 1 : p);
}

__device__ __forceinline__ float head_gate(const LA& a, int r, int head) { return a.gate ? sigmoid_f32(a.gate[(size_t)r * a.H + head]) : 1.0f; }

// ------------------------------------------------------------------------------------------
// Norms of the two latents, and the row's cache entry.
// ------------------------------------------------------------------------------------------
template <typename T>
__global__ __launch_bounds__(256) void latent_append_kernel(LA a) {
  constexpr int U = 2;                                    // pieces of eight features a thread holds (more: read again)
  __shared__ float red[2][4];
  const int r = blockIdx.x, Qp = (a.q_rank + 7) & ~7, own = a.kv_norm != nullptr;
  const T* p = reinterpret_cast<const T*>(a.proj) + (size_t)r * a.ld;
  const T* c = p + Qp;
  const int pos = position_of(a, r);
  const float* cs = a.cos_sin + (size_t)pos * a.P;
  const int nq = Qp / 8, nc = a.R / 8, np = own ? a.P / 8 : 0, rot_at = 255 - (int)threadIdx.x;     // (the last threads turn the rotated part)
  // everything is requested before the first sum: latents, norms' weights, angles (padding columns of proj are zero)
  float v[U][8], w[U][8], l[8], lw[8], t[8];
#pragma unroll
  for (int u = 0; u < U; ++u) {
    const int i = threadIdx.x + u * 256 < nq ? threadIdx.x + u * 256 : 0;
    load8(p + i * 8, true, 8, v[u]);
    load8(a.q_norm + i * 8, i * 8 + 8 <= a.q_rank, a.q_rank - i * 8, w[u]);
  }
  const int lc = threadIdx.x < nc ? threadIdx.x : 0, rc = rot_at < np ? rot_at : 0;
  if (own) {
    load8(c + lc * 8, true, 8, l);
    load8(a.kv_norm + lc * 8, lc * 8 + 8 <= a.kv_rank, a.kv_rank - lc * 8, lw);
    load8(c + a.R + rc * 8, true, 8, t);
    rotate8(cs + rc * 8, t);
  }
  float sq = 0.f, sc = 0.f;
#pragma unroll
  for (int u = 0; u < U; ++u)
    if (threadIdx.x + u * 256 < nq)
#pragma unroll
      for (int e = 0; e < 8; ++e) sq = __builtin_fmaf(v[u][e], v[u][e], sq);
  for (int i = threadIdx.x + U * 256; i < nq; i += 256) {
    float y[8];
    load8(p + i * 8, true, 8, y);
#pragma unroll
    for (int e = 0; e < 8; ++e) sq = __builtin_fmaf(y[e], y[e], sq);
  }
  if (own && threadIdx.x < nc)
#pragma unroll
    for (int e = 0; e < 8; ++e) sc = __builtin_fmaf(l[e], l[e], sc);
  sq = wave_total_dpp(sq);
  sc = wave_total_dpp(sc);
  if ((threadIdx.x & 63) == 0) {
    red[0][threadIdx.x >> 6] = sq;
    red[1][threadIdx.x >> 6] = sc;
  }
  __syncthreads();
  const float iq = 1.0f / sqrtf((red[0][0] + red[0][1] + red[0][2] + red[0][3]) / (float)a.q_rank + a.eps);
  T* cq = reinterpret_cast<T*>(a.cq) + (size_t)r * Qp;
#pragma unroll
  for (int u = 0; u < U; ++u) {
    const int i = threadIdx.x + u * 256;
    if (i >= nq) break;
#pragma unroll
    for (int e = 0; e < 8; ++e) v[u][e] = v[u][e] * iq * w[u][e];
    store8(cq + i * 8, v[u]);
  }
  for (int i = threadIdx.x + U * 256; i < nq; i += 256) {
    float y[8], yw[8];
    load8(p + i * 8, true, 8, y);
    load8(a.q_norm + i * 8, i * 8 + 8 <= a.q_rank, a.q_rank - i * 8, yw);
#pragma unroll
    for (int e = 0; e < 8; ++e) y[e] = y[e] * iq * yw[e];
    store8(cq + i * 8, y);
  }
  if (!own) return;
  const float ic = 1.0f / sqrtf((red[1][0] + red[1][1] + red[1][2] + red[1][3]) / (float)a.kv_rank + a.eps);
  T* dst = reinterpret_cast<T*>(a.ring) + ((size_t)a.slot[r] * a.ring_len + pos % a.ring_len) * (a.R + a.P);
  if (threadIdx.x < nc) {
#pragma unroll
    for (int e = 0; e < 8; ++e) l[e] = l[e] * ic * lw[e];
    store8(dst + lc * 8, l);
  }
  if (rot_at < np) store8(dst + a.R + rc * 8, t);
}

// ------------------------------------------------------------------------------------------
// Queries against the latent: W_uk,h^T q_h, and the rotated part behind it.
// ------------------------------------------------------------------------------------------
// 16 rows and 64 channels of one head per workgroup, 16 channels per wave
__global__ __launch_bounds__(256) void latent_absorb_kernel(LA a, int blocks) {
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, lg = lane >> 4, lc = lane & 15;
  const int head = blockIdx.x / blocks, nb = blockIdx.x % blocks, r0 = blockIdx.y * 16;
  const int RS = a.R + a.P, QD = a.D + a.P;
  const bf16* qb = reinterpret_cast<const bf16*>(a.q);
  bf16* out = reinterpret_cast<bf16*>(a.q_latent);
  const int n0 = nb * 64 + wave * 16, row = r0 + lc < a.rows ? r0 + lc : a.rows - 1;
  if (n0 < a.R) {                                         // (R is a multiple of 32: whole groups of 16 channels)
    const bf16* w = reinterpret_cast<const bf16*>(a.uk_t) + ((size_t)head * a.R + n0 + lc) * a.D + lg * 8;
    const bf16* q = qb + ((size_t)row * a.H + head) * QD + lg * 8;
    f32x4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll 4
    for (int k = 0; k < a.D; k += 32) acc = mma(*reinterpret_cast<const bf16x8*>(w + k), *reinterpret_cast<const bf16x8*>(q + k), acc);
    if (r0 + lc < a.rows) {
      bf16x4 y;
#pragma unroll
      for (int e = 0; e < 4; ++e) y[e] = (bf16)acc[e];
      *reinterpret_cast<bf16x4*>(out + ((size_t)row * a.H + head) * RS + n0 + lg * 4) = y;
    }
  }
  if (nb == 0) {
    const int pieces = a.P / 8;
    for (int i = threadIdx.x; i < 16 * pieces; i += 256) {
      const int r = r0 + i / pieces, f = (i % pieces) * 8;
      if (r >= a.rows) continue;
      float v[8];
      load8(qb + ((size_t)r * a.H + head) * QD + a.D + f, true, 8, v);
      rotate8(a.cos_sin + (size_t)position_of(a, r) * a.P + f, v);
      store8(out + ((size_t)r * a.H + head) * RS + a.R + f, v);
    }
  }
}

// a workgroup per (row, head)
__global__ __launch_bounds__(256) void latent_absorb_f32_kernel(LA a) {
  extern __shared__ __align__(16) float q_row[];
  const int r = blockIdx.x, head = blockIdx.y, RS = a.R + a.P;
  const float* q = reinterpret_cast<const float*>(a.q) + ((size_t)r * a.H + head) * (a.D + a.P);
  float* out = reinterpret_cast<float*>(a.q_latent) + ((size_t)r * a.H + head) * RS;
  for (int i = threadIdx.x; i < a.D; i += 256) q_row[i] = q[i];
  __syncthreads();
  for (int n = threadIdx.x; n < a.R; n += 256) {
    const float* w = reinterpret_cast<const float*>(a.uk_t) + ((size_t)head * a.R + n) * a.D;
    float s = 0.f;
    for (int k = 0; k < a.D; k += 4) {
      const f32x4 wv = *reinterpret_cast<const f32x4*>(w + k), qv = *reinterpret_cast<const f32x4*>(q_row + k);
#pragma unroll
      for (int e = 0; e < 4; ++e) s = __builtin_fmaf(wv[e], qv[e], s);
    }
    out[n] = s;
  }
  const float* cs = a.cos_sin + (size_t)position_of(a, r) * a.P;
  for (int i = threadIdx.x; i < a.P / 2; i += 256) {
    const float x = q[a.D + 2 * i], y = q[a.D + 2 * i + 1];
    out[a.R + 2 * i] = x * cs[2 * i] - y * cs[2 * i + 1];
    out[a.R + 2 * i + 1] = y * cs[2 * i] + x * cs[2 * i + 1];
  }
}

// the keys [j0, j1) of one part of a row's window
struct Part { int slot, j0, j1; };
__device__ __forceinline__ Part part_of(const LA& a, int r, int split) {
  const int i = position_of(a, r), lo = i - a.window + 1 > 0 ? i - a.window + 1 : 0;
  const int per = (i - lo + a.splits) / a.splits;
  const int j0 = lo + split * per, j1 = j0 + per < i + 1 ? j0 + per : i + 1;
  return Part{a.slot[r], j0, j1};
}

// ------------------------------------------------------------------------------------------
// Rows over the cache, bf16: a workgroup per (row, 16 heads, part of the window).  64 keys at a time lie in LDS as they are
// in the cache; a wave scores 16 of them against the 16 heads (S^T = K Q^T) and sums NT blocks of 16 latent features over
// all 64 (O^T = C^T P^T, C^T by transposed reads of the same rows).
// ------------------------------------------------------------------------------------------
constexpr int LR_KEYS = 64;
constexpr int LR_PS = LR_KEYS + 8;

static size_t latent_rows_smem(int RS) { return ((size_t)(LR_KEYS + 16) * (RS + 8) + 16 * LR_PS) * sizeof(bf16); }

template <int NT>
__global__ __launch_bounds__(256) void latent_rows_kernel(LA a, int groups) {
  constexpr int IT = NT * 2 + 4;                          // pieces of 16 bytes a thread moves per tile (R <= 64 NT, P <= 128)
  extern __shared__ __align__(16) bf16 tile[];
  __shared__ float wave_top[4][16], wave_sum_s[4][16];
  const int RS = a.R + a.P, KS = RS + 8;
  bf16* sk = tile;                                        // [64][KS]
  bf16* sq = sk + LR_KEYS * KS;                           // [16][KS]
  bf16* sp = sq + 16 * KS;                                // [16][LR_PS]
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, lg = lane >> 4, lc = lane & 15;
  int b = blockIdx.x;
  const int split = b % a.splits; b /= a.splits;
  const int hg = b % groups, r = b / groups;
  const Part part = part_of(a, r, split);
  const bf16* ring = reinterpret_cast<const bf16*>(a.ring) + (size_t)part.slot * a.ring_len * RS;
  const int steps = RS / 32;

  u32x4 pf[IT];
  const int my_key = threadIdx.x >> 2, my_piece = (threadIdx.x & 3) * 8;
  auto fetch = [&](int jt) {
    const int j = jt + my_key < part.j1 ? jt + my_key : part.j1 - 1;
    const bf16* src = ring + (size_t)(j % a.ring_len) * RS + my_piece;
#pragma unroll
    for (int it = 0; it < IT; ++it) pf[it] = *reinterpret_cast<const u32x4*>(src + (it < steps ? it : 0) * 32);
  };
  if (part.j0 < part.j1) fetch(part.j0);
  {
    const int h = hg * 16 + (threadIdx.x >> 4), hc = h < a.H ? h : a.H - 1;
    const bf16* q = reinterpret_cast<const bf16*>(a.q_latent) + ((size_t)r * a.H + hc) * RS;
    for (int c = (threadIdx.x & 15) * 8; c < RS; c += 128)
      *reinterpret_cast<u32x4*>(sq + (threadIdx.x >> 4) * KS + c) = *reinterpret_cast<const u32x4*>(q + c);
  }

  f32x4 o[NT];
  float m = -1e30f, l = 0.f;                              // of head lc; l: this lane's share
#pragma unroll
  for (int t = 0; t < NT; ++t) o[t] = f32x4{0.f, 0.f, 0.f, 0.f};
  for (int jt = part.j0; jt < part.j1; jt += LR_KEYS) {
    __syncthreads();
#pragma unroll
    for (int it = 0; it < IT; ++it)
      if (it < steps) *reinterpret_cast<u32x4*>(sk + my_key * KS + it * 32 + my_piece) = pf[it];
    __syncthreads();
    if (jt + LR_KEYS < part.j1) fetch(jt + LR_KEYS);
    f32x4 s = {0.f, 0.f, 0.f, 0.f}, s2 = {0.f, 0.f, 0.f, 0.f};
    const bf16* kr = sk + (wave * 16 + lc) * KS + lg * 8;
    const bf16* qr = sq + lc * KS + lg * 8;
    int c = 0;
#pragma unroll 2
    for (; c + 2 <= steps; c += 2) {
      s = mma(*reinterpret_cast<const bf16x8*>(kr + c * 32), *reinterpret_cast<const bf16x8*>(qr + c * 32), s);
      s2 = mma(*reinterpret_cast<const bf16x8*>(kr + c * 32 + 32), *reinterpret_cast<const bf16x8*>(qr + c * 32 + 32), s2);
    }
    if (c < steps) s = mma(*reinterpret_cast<const bf16x8*>(kr + c * 32), *reinterpret_cast<const bf16x8*>(qr + c * 32), s);
    float top = -1e30f;
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      s[e] = jt + wave * 16 + lg * 4 + e < part.j1 ? (s[e] + s2[e]) * a.scale : -INFINITY;
      top = fmaxf(top, s[e]);
    }
    top = fmaxf(top, __shfl_xor(top, 16, 64));
    top = fmaxf(top, __shfl_xor(top, 32, 64));
    if (lane < 16) wave_top[wave][lc] = top;
    __syncthreads();
    top = m;
#pragma unroll
    for (int w = 0; w < 4; ++w) top = fmaxf(top, wave_top[w][lc]);
    const float keep = __expf(m - top);
    m = top;
    bf16x4 p;
    float sum = 0.f;
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const float x = __expf(s[e] - top);
      sum += x;
      p[e] = (bf16)x;
    }
    l = l * keep + sum;
    *reinterpret_cast<bf16x4*>(sp + lc * LR_PS + wave * 16 + lg * 4) = p;
    __syncthreads();
#pragma unroll
    for (int t = 0; t < NT; ++t)
#pragma unroll
      for (int e = 0; e < 4; ++e) o[t][e] *= keep;
#pragma unroll
    for (int kg = 0; kg < LR_KEYS / 32; ++kg) {
      const bf16x8 pb = *reinterpret_cast<const bf16x8*>(sp + lc * LR_PS + kg * 32 + lg * 8);
      const bf16* v = sk + (kg * 32 + lg * 8 + (lc >> 2)) * KS + (lc & 3) * 4;
#pragma unroll
      for (int t = 0; t < NT; ++t) {
        const int d0 = (wave * NT + t) * 16;
        if (d0 < a.R) o[t] = mma(join(read_transposed(v + d0), read_transposed(v + d0 + 4 * KS)), pb, o[t]);
      }
    }
  }
  l += __shfl_xor(l, 16, 64);
  l += __shfl_xor(l, 32, 64);
  if (lane < 16) wave_sum_s[wave][lc] = l;
  __syncthreads();
  const int h = hg * 16 + lc;
  if (h >= a.H) return;
  const size_t at = ((size_t)r * a.H + h) * a.splits + split;
#pragma unroll
  for (int t = 0; t < NT; ++t) {
    const int d0 = (wave * NT + t) * 16;
    if (d0 < a.R) *reinterpret_cast<f32x4*>(a.part_o + at * a.R + d0 + lg * 4) = o[t];
  }
  if (threadIdx.x < 16) {
    a.part_ml[at * 2] = m;
    a.part_ml[at * 2 + 1] = wave_sum_s[0][lc] + wave_sum_s[1][lc] + wave_sum_s[2][lc] + wave_sum_s[3][lc];
  }
}

// Any size and type on the vector unit: a workgroup per (row, head, part); four lanes per key.
constexpr int LV_FEATURES = 8;           // latent features of a thread: R <= 2048

template <typename T>
__global__ __launch_bounds__(256) void latent_rows_vector_kernel(LA a) {
  extern __shared__ __align__(16) float q_row[];
  __shared__ float score[64], weight[64];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, RS = a.R + a.P;
  int b = blockIdx.x;
  const int split = b % a.splits; b /= a.splits;
  const int head = b % a.H, r = b / a.H;
  const Part part = part_of(a, r, split);
  const T* ring = reinterpret_cast<const T*>(a.ring) + (size_t)part.slot * a.ring_len * RS;
  const T* q = reinterpret_cast<const T*>(a.q_latent) + ((size_t)r * a.H + head) * RS;
  for (int c = threadIdx.x; c < RS; c += 256) q_row[c] = (float)q[c];
  float o[LV_FEATURES], m = -1e30f, l = 0.f;
#pragma unroll
  for (int n = 0; n < LV_FEATURES; ++n) o[n] = 0.f;
  for (int jt = part.j0; jt < part.j1; jt += 64) {
    __syncthreads();
    const int key = threadIdx.x >> 2, sub = (threadIdx.x & 3) * 8;
    const int j = jt + key < part.j1 ? jt + key : part.j1 - 1;
    const T* k = ring + (size_t)(j % a.ring_len) * RS;
    float t = 0.f;
    for (int c = sub; c < RS; c += 32) {
      float v[8];
      load8(k + c, true, 8, v);
#pragma unroll
      for (int e = 0; e < 8; ++e) t = __builtin_fmaf(v[e], q_row[c + e], t);
    }
    t += __shfl_xor(t, 1, 64);
    t += __shfl_xor(t, 2, 64);
    if ((threadIdx.x & 3) == 0) score[key] = jt + key < part.j1 ? t * a.scale : -INFINITY;
    __syncthreads();
    const float s = score[lane], top = fmaxf(m, wave_max(s)), p = expf(s - top), keep = expf(m - top);
    l = l * keep + wave_sum(p);
    m = top;
    if (wave == 0) weight[lane] = p;
    __syncthreads();
    const int n_keys = part.j1 - jt < 64 ? part.j1 - jt : 64;
#pragma unroll
    for (int n = 0; n < LV_FEATURES; ++n) {
      const int c = threadIdx.x + n * 256;
      if (c >= a.R) break;
      float x = o[n] * keep;
      for (int u = 0; u < n_keys; ++u) x = __builtin_fmaf(weight[u], (float)ring[(size_t)((jt + u) % a.ring_len) * RS + c], x);
      o[n] = x;
    }
  }
  const size_t at = ((size_t)r * a.H + head) * a.splits + split;
#pragma unroll
  for (int n = 0; n < LV_FEATURES; ++n) {
    const int c = threadIdx.x + n * 256;
    if (c < a.R) a.part_o[at * a.R + c] = o[n];
  }
  if (threadIdx.x == 0) {
    a.part_ml[at * 2] = m;
    a.part_ml[at * 2 + 1] = l;
  }
}

// ------------------------------------------------------------------------------------------
// The parts of a row meet, and each head's W_uv and gate are applied.
// ------------------------------------------------------------------------------------------
// the weights of one row's parts (lane = part), each divided by the sum of all softmax weights
__device__ __forceinline__ float part_weight(const LA& a, int r, int head, int lane) {
  float m = -1e30f, l = 0.f;
  if (lane < a.splits) {
    const float* ml = a.part_ml + (((size_t)r * a.H + head) * a.splits + lane) * 2;
    m = ml[0];
    l = ml[1];
  }
  const float top = wave_max(m), w = lane < a.splits ? expf(m - top) : 0.f;
  return w / wave_sum(w * l);
}

// Up to 16 rows (`each`) and NB * 16 value channels of one head per workgroup.  The parts meet first: 16 lanes take 128 latent
// features of a row, and the weighted sums go to LDS, where the waves share the latent features of the product.
template <int NB>
__global__ __launch_bounds__(256) void latent_values_kernel(LA a, int blocks, int each) {
  constexpr int AHEAD = 4;                                // steps of the product whose weights are requested at the start
  extern __shared__ __align__(16) bf16 xs[];              // [16][R + 8]
  __shared__ float weight[16][64];
  __shared__ f32x4 red[4][NB][64];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, lg = lane >> 4, lc = lane & 15, XS = a.R + 8;
  const int head = blockIdx.x / blocks, n0 = (blockIdx.x % blocks) * NB * 16, r0 = blockIdx.y * each;
  const int count = a.rows - r0 < each ? a.rows - r0 : each, row = r0 + (lc < count ? lc : count - 1);
  const bf16* w[NB];
  bf16x8 wv[AHEAD][NB];
#pragma unroll
  for (int n = 0; n < NB; ++n) {
    const int ch = n0 + n * 16 + lc;
    w[n] = reinterpret_cast<const bf16*>(a.uv) + ((size_t)head * a.E + (ch < a.E ? ch : a.E - 1)) * a.R + lg * 8;
#pragma unroll
    for (int i = 0; i < AHEAD; ++i) {
      const int k = wave * 32 + i * 128;
      wv[i][n] = *reinterpret_cast<const bf16x8*>(w[n] + (k < a.R ? k : 0));
    }
  }
  for (int n = wave; n < count; n += 4) weight[n][lane] = part_weight(a, r0 + n, head, lane);
  __syncthreads();
  const int chunks = (a.R + 127) / 128, units = count * chunks;
  for (int u = wave * 4 + lg; u < units; u += 16) {
    const int n = u / chunks, c = (u % chunks) * 128 + lc * 8;
    if (c >= a.R) continue;
    const float* po = a.part_o + ((size_t)(r0 + n) * a.H + head) * a.splits * a.R + c;
    float x[8] = {};
    int s = 0;
    for (; s + 8 <= a.splits; s += 8) {
      float v[8][8];
#pragma unroll
      for (int i = 0; i < 8; ++i) load8(po + (size_t)(s + i) * a.R, true, 8, v[i]);
#pragma unroll
      for (int i = 0; i < 8; ++i) {
        const float f = weight[n][s + i];
#pragma unroll
        for (int e = 0; e < 8; ++e) x[e] = __builtin_fmaf(f, v[i][e], x[e]);
      }
    }
    for (; s < a.splits; ++s) {
      float v[8];
      load8(po + (size_t)s * a.R, true, 8, v);
      const float f = weight[n][s];
#pragma unroll
      for (int e = 0; e < 8; ++e) x[e] = __builtin_fmaf(f, v[e], x[e]);
    }
    store8(xs + n * XS + c, x);
  }
  __syncthreads();
  f32x4 acc[NB];
#pragma unroll
  for (int n = 0; n < NB; ++n) acc[n] = f32x4{0.f, 0.f, 0.f, 0.f};
  const bf16* xr = xs + (lc < count ? lc : count - 1) * XS + lg * 8;
#pragma unroll
  for (int i = 0; i < AHEAD; ++i) {
    const int k = wave * 32 + i * 128;
    if (k >= a.R) break;
    const bf16x8 xb = *reinterpret_cast<const bf16x8*>(xr + k);
#pragma unroll
    for (int n = 0; n < NB; ++n) acc[n] = mma(wv[i][n], xb, acc[n]);
  }
  for (int k = wave * 32 + AHEAD * 128; k < a.R; k += 128) {
    const bf16x8 xb = *reinterpret_cast<const bf16x8*>(xr + k);
#pragma unroll
    for (int n = 0; n < NB; ++n) acc[n] = mma(*reinterpret_cast<const bf16x8*>(w[n] + k), xb, acc[n]);
  }
#pragma unroll
  for (int n = 0; n < NB; ++n) red[wave][n][lane] = acc[n];
  __syncthreads();
  if (wave >= NB || lc >= count) return;
  const int ch = n0 + wave * 16 + lg * 4;
  if (ch >= a.E) return;
  f32x4 y = red[0][wave][lane];
#pragma unroll
  for (int v = 1; v < 4; ++v) {
    const f32x4 t = red[v][wave][lane];
#pragma unroll
    for (int e = 0; e < 4; ++e) y[e] += t[e];
  }
  const float g = head_gate(a, row, head);
  if (a.feature_gate) {
    const bf16x4 fg = *reinterpret_cast<const bf16x4*>(reinterpret_cast<const bf16*>(a.feature_gate) + (size_t)row * a.gate_ld + head * a.E + ch);
#pragma unroll
    for (int e = 0; e < 4; ++e) y[e] *= sigmoid_f32((float)fg[e]);
  }
  bf16x4 yb;
#pragma unroll
  for (int e = 0; e < 4; ++e) yb[e] = (bf16)(y[e] * g);
  *reinterpret_cast<bf16x4*>(reinterpret_cast<bf16*>(a.out) + ((size_t)row * a.H + head) * a.E + ch) = yb;
}

// a workgroup per (row, head), a wave per channel
template <typename T>
__global__ __launch_bounds__(256) void latent_values_vector_kernel(LA a) {
  extern __shared__ __align__(16) float x_row[];
  __shared__ float weight[64];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, r = blockIdx.x, head = blockIdx.y;
  const float mine = part_weight(a, r, head, lane);
  if (wave == 0) weight[lane] = mine;
  __syncthreads();
  const float* po = a.part_o + ((size_t)r * a.H + head) * a.splits * a.R;
  for (int c = threadIdx.x; c < a.R; c += 256) {
    float x = 0.f;
    for (int s = 0; s < a.splits; ++s) x = __builtin_fmaf(weight[s], po[(size_t)s * a.R + c], x);
    x_row[c] = (float)(T)x;
  }
  __syncthreads();
  const float g = head_gate(a, r, head);
  const T* fg = a.feature_gate ? reinterpret_cast<const T*>(a.feature_gate) + (size_t)r * a.gate_ld + head * a.E : nullptr;
  for (int n = wave; n < a.E; n += 4) {
    const T* w = reinterpret_cast<const T*>(a.uv) + ((size_t)head * a.E + n) * a.R;
    float s = 0.f;
    for (int c = lane; c < a.R; c += 64) s = __builtin_fmaf((float)w[c], x_row[c], s);
    s = wave_sum(s);
    if (lane == 0) reinterpret_cast<T*>(a.out)[((size_t)r * a.H + head) * a.E + n] = (T)(fg ? s * g * sigmoid_f32((float)fg[n]) : s * g);
  }
}

// ------------------------------------------------------------------------------------------
// Cache rows side by side: the latents, and the rotated parts
// ------------------------------------------------------------------------------------------
__global__ __launch_bounds__(256) void latent_gather_kernel(LA a, int pieces, int latent_pieces) {
  const size_t idx = (size_t)blockIdx.x * 256 + threadIdx.x;
  const size_t key = idx / pieces;
  if (key >= (size_t)a.keys) return;
  const int c = (int)(idx % pieces);
  const u32x4* ring = reinterpret_cast<const u32x4*>(a.ring);
  const u32x4 v = ring[((size_t)a.key_slot[key] * a.ring_len + a.key_pos[key] % a.ring_len) * pieces + c];
  if (c < latent_pieces) reinterpret_cast<u32x4*>(a.key_latent)[key * latent_pieces + c] = v;
  else reinterpret_cast<u32x4*>(a.key_rot)[key * (pieces - latent_pieces) + c - latent_pieces] = v;
}

// ------------------------------------------------------------------------------------------
// Many rows over per-head keys and values (bf16): a workgroup of four waves takes up to 128 rows of one head, a wave 2
// groups of 16; 64 keys at a time pass through LDS.  S^T = K Q^T, O^T = V^T P^T.  A lane holds scores of ONE query, keys
// 16 t + 4 (lane / 16) + 0..3 of every 16-key group t; two groups are the eight values of a B operand as they stand, and
// the transposed reads of V take the keys in that order.
// ------------------------------------------------------------------------------------------
constexpr int LT_KEYS = 64;

template <int DKT, int DVT>
__global__ __launch_bounds__(256) void latent_tile_kernel(LA a) {
  constexpr int QW = 2, KS = DKT * 32 + 8, VS = DVT * 16 + 8, VIT = (DVT + 1) / 2;
  __shared__ __align__(16) bf16 sk[LT_KEYS * KS];
  __shared__ __align__(16) bf16 sv[LT_KEYS * (VIT * 32 + 8)];
  static_assert(VS == VIT * 32 + 8, "value blocks come in pairs");
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, lg = lane >> 4, lc = lane & 15;
  const int head = blockIdx.x, tile = blockIdx.y;
  const int D = a.D, QD = a.D + a.P, E = a.E, ld = a.H * (D + E);
  const int count = a.tile_count[tile], row0 = a.tile_row[tile], key0 = a.tile_key[tile];
  const int p0 = position_of(a, row0);
  const bf16* kb = reinterpret_cast<const bf16*>(a.kv) + head * D;
  const bf16* vb = reinterpret_cast<const bf16*>(a.kv) + a.H * D + head * E;
  const bf16* rb = reinterpret_cast<const bf16*>(a.key_rot);

  // queries: lane holds features 32 m + 8 lg + 0..7 of row lc of each of its groups
  bf16x8 qf[QW][DKT];
  int qi[QW];
#pragma unroll
  for (int w = 0; w < QW; ++w) {
    int n = (wave * QW + w) * 16 + lc;
    qi[w] = p0 + n;
    n = n < count ? n : count - 1;
    const bf16* q = reinterpret_cast<const bf16*>(a.q) + ((size_t)(row0 + n) * a.H + head) * QD + lg * 8;
    const float* cs = a.cos_sin + (size_t)position_of(a, row0 + n) * a.P + lg * 8;
#pragma unroll
    for (int m = 0; m < DKT; ++m) {
      if (m * 32 < D) {
        qf[w][m] = *reinterpret_cast<const bf16x8*>(q + m * 32);
      } else if (m * 32 < QD) {
        float v[8];
        load8(q + m * 32, true, 8, v);
        rotate8(cs + m * 32 - D, v);
#pragma unroll
        for (int e = 0; e < 8; ++e) qf[w][m][e] = (bf16)v[e];
      } else {
#pragma unroll
        for (int e = 0; e < 8; ++e) qf[w][m][e] = (bf16)0.0f;
      }
    }
  }
  const int i_last = p0 + count - 1;
  const int lo = p0 - a.window + 1 > 0 ? p0 - a.window + 1 : 0;
  const int w_first = p0 + wave * QW * 16, w_last = w_first + QW * 16 - 1;
  const float scale2 = a.scale * 1.4426950408889634f;

  u32x4 kf[DKT], vf[VIT];
  const int my_key = threadIdx.x >> 2, my_piece = (threadIdx.x & 3) * 8;
  auto fetch = [&](int jt) {
    const int j = jt + my_key < i_last ? jt + my_key : i_last;
    const bf16* k = kb + (size_t)(key0 + j) * ld + my_piece;
    const bf16* v = vb + (size_t)(key0 + j) * ld;
    const bf16* rot = rb + (size_t)(key0 + j) * a.P + my_piece;
#pragma unroll
    for (int m = 0; m < DKT; ++m) kf[m] = *reinterpret_cast<const u32x4*>(m * 32 < D ? k + m * 32 : rot + (m * 32 < QD ? m * 32 - D : 0));
#pragma unroll
    for (int m = 0; m < VIT; ++m) vf[m] = *reinterpret_cast<const u32x4*>(v + (m * 32 + my_piece < E ? m * 32 + my_piece : 0));
  };
  f32x4 o[QW][DVT];
  float mx[QW], l[QW];
#pragma unroll
  for (int w = 0; w < QW; ++w) {
    mx[w] = -1e30f;
    l[w] = 0.f;
#pragma unroll
    for (int t = 0; t < DVT; ++t) o[w][t] = f32x4{0.f, 0.f, 0.f, 0.f};
  }
  fetch(lo);
  for (int jt = lo; jt <= i_last; jt += LT_KEYS) {
    __syncthreads();
#pragma unroll
    for (int m = 0; m < DKT; ++m) *reinterpret_cast<u32x4*>(sk + my_key * KS + m * 32 + my_piece) = kf[m];
#pragma unroll
    for (int m = 0; m < VIT; ++m) *reinterpret_cast<u32x4*>(sv + my_key * VS + m * 32 + my_piece) = vf[m];
    __syncthreads();
    if (jt + LT_KEYS <= i_last) fetch(jt + LT_KEYS);
    if (jt > w_last || jt + LT_KEYS - 1 < w_first - a.window + 1) continue;       // nothing this wave's rows see
    f32x4 s[QW][4];
#pragma unroll
    for (int t = 0; t < 4; ++t) {
#pragma unroll
      for (int w = 0; w < QW; ++w) s[w][t] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int c = 0; c < DKT; ++c) {
        const bf16x8 kv = *reinterpret_cast<const bf16x8*>(sk + (t * 16 + lc) * KS + c * 32 + lg * 8);
#pragma unroll
        for (int w = 0; w < QW; ++w) s[w][t] = mma(kv, qf[w][c], s[w][t]);
      }
    }
    bf16x8 p[QW][2];
#pragma unroll
    for (int w = 0; w < QW; ++w) {
      float top = mx[w];
#pragma unroll
      for (int t = 0; t < 4; ++t)
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          const int dist = qi[w] - (jt + t * 16 + lg * 4 + e);
          s[w][t][e] = dist >= 0 && dist < a.window ? s[w][t][e] * scale2 : -INFINITY;
          top = fmaxf(top, s[w][t][e]);
        }
      top = fmaxf(top, __shfl_xor(top, 16, 64));
      top = fmaxf(top, __shfl_xor(top, 32, 64));
      const float keep = exp2f(mx[w] - top);
      mx[w] = top;
      float sum = 0.f;
#pragma unroll
      for (int t = 0; t < 4; ++t)
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          const float x = exp2f(s[w][t][e] - top);
          sum += x;
          p[w][t >> 1][(t & 1) * 4 + e] = (bf16)x;
        }
      l[w] = l[w] * keep + sum;
#pragma unroll
      for (int t = 0; t < DVT; ++t)
#pragma unroll
        for (int e = 0; e < 4; ++e) o[w][t][e] *= keep;
    }
#pragma unroll
    for (int kg = 0; kg < 2; ++kg) {
      const bf16* v = sv + (kg * 32 + lg * 4 + (lc >> 2)) * VS + (lc & 3) * 4;
#pragma unroll
      for (int t = 0; t < DVT; ++t) {
        const bf16x8 vt = join(read_transposed(v + t * 16), read_transposed(v + t * 16 + 16 * VS));
#pragma unroll
        for (int w = 0; w < QW; ++w) o[w][t] = mma(vt, p[w][kg], o[w][t]);
      }
    }
  }
#pragma unroll
  for (int w = 0; w < QW; ++w) {
    float tot = l[w];
    tot += __shfl_xor(tot, 16, 64);
    tot += __shfl_xor(tot, 32, 64);
    const int n = (wave * QW + w) * 16 + lc;
    if (n >= count) continue;
    const float f = head_gate(a, row0 + n, head) / tot;
    const bf16* fg = a.feature_gate ? reinterpret_cast<const bf16*>(a.feature_gate) + (size_t)(row0 + n) * a.gate_ld + head * E : nullptr;
    bf16* out = reinterpret_cast<bf16*>(a.out) + ((size_t)(row0 + n) * a.H + head) * E;
#pragma unroll
    for (int t = 0; t < DVT; ++t) {
      if (t * 16 >= E) break;
      bf16x4 y;
      if (fg) {
        const bf16x4 gv = *reinterpret_cast<const bf16x4*>(fg + t * 16 + lg * 4);
#pragma unroll
        for (int e = 0; e < 4; ++e) y[e] = (bf16)(o[w][t][e] * f / (1.0f + __expf(-(float)gv[e])));
      } else {
#pragma unroll
        for (int e = 0; e < 4; ++e) y[e] = (bf16)(o[w][t][e] * f);
      }
      *reinterpret_cast<bf16x4*>(out + t * 16 + lg * 4) = y;
    }
  }
}

// ------------------------------------------------------------------------------------------
static int check_latent(const LA& a, const char* name) {
  PTA_REQUIRE(a.dtype == PTA_BF16 || a.dtype == PTA_FP32, "%s: unknown type %d", name, a.dtype);
  PTA_REQUIRE(a.rows > 0 && a.H > 0 && a.H <= 65535, "%s: rows %d, heads %d", name, a.rows, a.H);
  PTA_REQUIRE(a.D > 0 && a.D % 32 == 0 && a.P > 0 && a.P % 32 == 0 && a.R > 0 && a.R % 32 == 0 && a.E > 0 && a.E % 16 == 0,
              "%s: sizes D %d, P %d, R %d must be multiples of 32 and E %d of 16", name, a.D, a.P, a.R, a.E);
  PTA_REQUIRE(a.R <= 256 * LV_FEATURES && a.R + a.P <= 16000 && a.D <= 16000, "%s: latent of %d (at most %d)", name, a.R, 256 * LV_FEATURES);
  PTA_REQUIRE(!a.feature_gate || (pta_aligned(a.feature_gate, 16) && a.gate_ld % 8 == 0 && a.gate_ld >= a.H * a.E), "%s: unaligned gate, or rows of %d",
              name, a.gate_ld);
  PTA_REQUIRE(a.cos_sin && a.positions > 0 && a.ring && pta_aligned(a.ring, 16) && a.ring_len > 0 && a.slot && a.pos,
              "%s: positions, the cache or the rows' places are missing", name);
  return PTA_OK;
}

#define LATENT_ENTRY(name)                              \
  PTA_REQUIRE(args, name ": null arguments");           \
  const LA& a = *args;                                  \
  {                                                     \
    const int rc = check_latent(a, name);               \
    if (rc) return rc;                                  \
  }                                                     \
  hipStream_t s = (hipStream_t)stream;

extern "C" int pta_latent_append(const LA* args, pta_stream_t stream) {
  LATENT_ENTRY("pta_latent_append")
  const int Qp = (a.q_rank + 7) & ~7;
  PTA_REQUIRE(a.proj && a.q_norm && a.cq && a.q_rank > 0, "pta_latent_append: null pointer, or query latent of %d", a.q_rank);
  PTA_REQUIRE(a.ld >= Qp + (a.kv_norm ? a.R + a.P : 0), "pta_latent_append: rows of %d do not hold the latents", a.ld);
  PTA_REQUIRE(!a.kv_norm || (a.kv_rank > 0 && a.kv_rank <= a.R && a.P <= 256 * 8), "pta_latent_append: latent of %d in %d, rotated part of %d",
              a.kv_rank, a.R, a.P);
  PTA_REQUIRE(a.ld % 8 == 0 && pta_aligned(a.proj, 16) && pta_aligned(a.cq, 16) && pta_aligned(a.q_norm, 16) &&
              (!a.kv_norm || pta_aligned(a.kv_norm, 16)), "pta_latent_append: unaligned operand");
  if (a.dtype == PTA_BF16) hipLaunchKernelGGL((latent_append_kernel<bf16>), dim3(a.rows), dim3(256), 0, s, a);
  else hipLaunchKernelGGL((latent_append_kernel<float>), dim3(a.rows), dim3(256), 0, s, a);
  PTA_CHECK_LAUNCH("pta_latent_append");
  return PTA_OK;
}

extern "C" int pta_latent_absorb(const LA* args, pta_stream_t stream) {
  LATENT_ENTRY("pta_latent_absorb")
  PTA_REQUIRE(a.q && a.uk_t && a.q_latent && pta_aligned(a.q, 16) && pta_aligned(a.uk_t, 16) && pta_aligned(a.q_latent, 16),
              "pta_latent_absorb: null or unaligned operand");
  if (a.dtype == PTA_BF16) {
    const int blocks = (a.R + 63) / 64;
    hipLaunchKernelGGL(latent_absorb_kernel, dim3(a.H * blocks, (a.rows + 15) / 16), dim3(256), 0, s, a, blocks);
  } else {
    hipLaunchKernelGGL(latent_absorb_f32_kernel, dim3(a.rows, a.H), dim3(256), a.D * sizeof(float), s, a);
  }
  PTA_CHECK_LAUNCH("pta_latent_absorb");
  return PTA_OK;
}

template <int NT>
static int launch_latent_rows(const LA& a, hipStream_t s) {
  const size_t smem = latent_rows_smem(a.R + a.P);
  const int groups = (a.H + 15) / 16;
  if (smem > 60 * 1024)
    PTA_REQUIRE(hipFuncSetAttribute((const void*)latent_rows_kernel<NT>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)smem) == hipSuccess,
                "pta_latent_rows: %zu bytes of LDS refused", smem);
  hipLaunchKernelGGL((latent_rows_kernel<NT>), dim3((unsigned)((size_t)a.rows * groups * a.splits)), dim3(256), smem, s, a, groups);
  return PTA_OK;
}

extern "C" int pta_latent_rows(const LA* args, pta_stream_t stream) {
  LATENT_ENTRY("pta_latent_rows")
  PTA_REQUIRE(a.q_latent && a.part_o && a.part_ml && a.window > 0 && a.splits >= 1 && a.splits <= 64,
              "pta_latent_rows: null pointer, window %d, or splits %d (1 .. 64)", a.window, a.splits);
  PTA_REQUIRE(pta_aligned(a.q_latent, 16) && pta_aligned(a.part_o, 16), "pta_latent_rows: unaligned operand");
  int rc = PTA_OK;
  if (a.dtype == PTA_BF16 && a.R <= 1024 && a.P <= 128 && latent_rows_smem(a.R + a.P) <= 158 * 1024) {
    if (a.R <= 64) rc = launch_latent_rows<1>(a, s);
    else if (a.R <= 128) rc = launch_latent_rows<2>(a, s);
    else if (a.R <= 256) rc = launch_latent_rows<4>(a, s);
    else if (a.R <= 512) rc = launch_latent_rows<8>(a, s);
    else rc = launch_latent_rows<16>(a, s);
  } else {
    const dim3 grid((unsigned)((size_t)a.rows * a.H * a.splits));
    const size_t smem = (size_t)(a.R + a.P) * sizeof(float);
    if (a.dtype == PTA_BF16) hipLaunchKernelGGL((latent_rows_vector_kernel<bf16>), grid, dim3(256), smem, s, a);
    else hipLaunchKernelGGL((latent_rows_vector_kernel<float>), grid, dim3(256), smem, s, a);
  }
  if (rc) return rc;
  PTA_CHECK_LAUNCH("pta_latent_rows");
  return PTA_OK;
}

template <int NB>
static int launch_latent_values(const LA& a, int each, hipStream_t s) {
  const int blocks = (a.E + NB * 16 - 1) / (NB * 16);
  const size_t smem = (size_t)16 * (a.R + 8) * sizeof(bf16);        // (beside up to 20 KiB of fixed LDS)
  PTA_REQUIRE(smem <= 40 * 1024 || hipFuncSetAttribute((const void*)latent_values_kernel<NB>, hipFuncAttributeMaxDynamicSharedMemorySize,
                                                       (int)smem) == hipSuccess, "pta_latent_values: %zu bytes of LDS refused", smem);
  hipLaunchKernelGGL((latent_values_kernel<NB>), dim3(a.H * blocks, (a.rows + each - 1) / each), dim3(256), smem, s, a, blocks, each);
  return PTA_OK;
}

extern "C" int pta_latent_values(const LA* args, pta_stream_t stream) {
  LATENT_ENTRY("pta_latent_values")
  PTA_REQUIRE(a.part_o && a.part_ml && a.uv && a.out && a.splits >= 1 && a.splits <= 64,
              "pta_latent_values: null pointer, or splits %d (1 .. 64)", a.splits);
  PTA_REQUIRE(pta_aligned(a.part_o, 16) && pta_aligned(a.uv, 16) && pta_aligned(a.out, 16), "pta_latent_values: unaligned operand");
  if (a.dtype == PTA_BF16) {
    // few rows: many workgroups with few channels; a batch: fewer rows each, so that its parts are not read by too many
    const int rc = a.rows <= 4 ? launch_latent_values<2>(a, 16, s) : launch_latent_values<4>(a, a.rows <= 64 ? 4 : 16, s);
    if (rc) return rc;
  } else {
    hipLaunchKernelGGL((latent_values_vector_kernel<float>), dim3(a.rows, a.H), dim3(256), a.R * sizeof(float), s, a);
  }
  PTA_CHECK_LAUNCH("pta_latent_values");
  return PTA_OK;
}

extern "C" int pta_latent_gather(const LA* args, pta_stream_t stream) {
  LATENT_ENTRY("pta_latent_gather")
  PTA_REQUIRE(a.keys > 0 && a.key_slot && a.key_pos && a.key_latent && a.key_rot, "pta_latent_gather: null pointer, or %d keys", a.keys);
  PTA_REQUIRE(pta_aligned(a.key_latent, 16) && pta_aligned(a.key_rot, 16), "pta_latent_gather: unaligned buffer");
  const int es = a.dtype == PTA_BF16 ? 2 : 4, pieces = (a.R + a.P) * es / 16, latent = a.R * es / 16;
  hipLaunchKernelGGL(latent_gather_kernel, dim3((unsigned)(((size_t)a.keys * pieces + 255) / 256)), dim3(256), 0, s, a, pieces, latent);
  PTA_CHECK_LAUNCH("pta_latent_gather");
  return PTA_OK;
}

extern "C" int pta_latent_tiles_fit(int dtype, int D, int P, int E) { return dtype == PTA_BF16 && D + P <= 256 && E <= 256; }

template <int DKT>
static void launch_latent_tiles(const LA& a, hipStream_t s) {
  const dim3 grid(a.H, a.tiles);
  if (a.E <= 64) hipLaunchKernelGGL((latent_tile_kernel<DKT, 4>), grid, dim3(256), 0, s, a);
  else if (a.E <= 128) hipLaunchKernelGGL((latent_tile_kernel<DKT, 8>), grid, dim3(256), 0, s, a);
  else hipLaunchKernelGGL((latent_tile_kernel<DKT, 16>), grid, dim3(256), 0, s, a);
}

extern "C" int pta_latent_tiles(const LA* args, pta_stream_t stream) {
  LATENT_ENTRY("pta_latent_tiles")
  PTA_REQUIRE(pta_latent_tiles_fit(a.dtype, a.D, a.P, a.E), "pta_latent_tiles: bf16 with D + P and E up to 256");
  PTA_REQUIRE(a.q && a.kv && a.key_rot && a.out && a.window > 0, "pta_latent_tiles: null pointer, or window %d", a.window);
  PTA_REQUIRE(a.tile_row && a.tile_count && a.tile_key && a.tiles > 0 && a.tiles <= 65535, "pta_latent_tiles: %d tiles (1 .. 65535)", a.tiles);
  PTA_REQUIRE(pta_aligned(a.q, 16) && pta_aligned(a.kv, 16) && pta_aligned(a.key_rot, 16) && pta_aligned(a.out, 16),
              "pta_latent_tiles: unaligned operand");
  const int dk = a.D + a.P;
  if (dk <= 64) launch_latent_tiles<2>(a, s);
  else if (dk <= 128) launch_latent_tiles<4>(a, s);
  else if (dk <= 192) launch_latent_tiles<6>(a, s);
  else launch_latent_tiles<8>(a, s);
  PTA_CHECK_LAUNCH("pta_latent_tiles");
  return PTA_OK;
}
