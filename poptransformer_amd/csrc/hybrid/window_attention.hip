// Attention over a sliding window with a distance bias, whole-projection query / key norm, values that are the raw keys,
// and an output gate.
//
// The cache keeps one raw key row per token and key head, which is read once for both products, and the inverse root
// mean square of the token's keys; the key norm's weight, the query norm and the score scale are folded into the query:
//   score(i, j) = rinv_j * (q'_i . k_j) - slope * (i - j),   q' = q * rinv_q * w_q * w_k * scale.
#include "attention.h"

typedef pta_window_attention_args WA;

static __host__ __device__ inline int padded8(int d) { return (d + 7) & ~7; }

// this thread's share of the sum of squares of n consecutive elements (256 threads)
template <typename T>
__device__ __forceinline__ float squares(const T* p, int n, bool vec) {
  float s = 0.f, v[8];
  for (int c = threadIdx.x * 8; c < n; c += 2048) {
    load8(p + c, vec && c + 8 <= n, n - c, v);
#pragma unroll
    for (int e = 0; e < 8; ++e) s = __builtin_fmaf(v[e], v[e], s);
  }
  return s;
}

// key head g of a row into its ring row (Dp elements, zero past D)
template <typename T>
__device__ __forceinline__ void put_ring_row(const WA& a, const T* k, int g, int slot, int pos) {
  const int Dp = padded8(a.D);
  T* dst = reinterpret_cast<T*>(a.ring) + (((size_t)slot * a.G + g) * a.ring_len + pos % a.ring_len) * Dp;
  for (int c = threadIdx.x; c < Dp; c += blockDim.x) dst[c] = c < a.D ? k[g * a.D + c] : (T)0.0f;
}

template <typename T>
__global__ __launch_bounds__(256) void window_append_kernel(WA a, bool vec) {
  __shared__ float red[2][4];
  const int r = blockIdx.x;
  const T* q = reinterpret_cast<const T*>(a.q) + (size_t)r * a.ld;
  const T* k = reinterpret_cast<const T*>(a.k) + (size_t)r * a.ld;
  const float qs = workgroup_sum<4>(squares(q, a.H * a.D, vec), red[0]);
  const float ks = workgroup_sum<4>(squares(k, a.G * a.D, vec), red[1]);
  const int slot = a.slot[r], pos = a.pos[r];
  if (threadIdx.x == 0) {
    a.q_scale[r] = 1.0f / sqrtf(qs / (float)(a.H * a.D) + a.eps);
    a.rinv[(size_t)slot * a.ring_len + pos % a.ring_len] = 1.0f / sqrtf(ks / (float)(a.G * a.D) + a.eps);
  }
  for (int g = 0; g < a.G; ++g) put_ring_row(a, k, g, slot, pos);
}

// ------------------------------------------------------------------------------------------
// Row by row on the vector unit: a workgroup per (row, key head, up to RG of its query heads, part of the window).  LPK
// lanes share a key row (eight elements each), so a key is loaded once for the RG heads and for both products.
// FUSED: the row's own key comes from the projection and is put into the ring by this launch.
// ------------------------------------------------------------------------------------------
constexpr int WR_KEYS = 4;               // keys a lane group takes per step

template <typename T, int RG, int LPK>
__global__ __launch_bounds__(256) void window_rows_kernel(WA a, bool vec, int fused, int groups, float* part_o, float* part_ml) {
  constexpr int NG = 4 * 64 / LPK;       // lane groups of the workgroup, each with a softmax state of its own
  constexpr int DL = LPK * 8;
  __shared__ float red[2][4];
  __shared__ float sm[NG][RG], sl[NG][RG];
  __shared__ __align__(16) float so[NG * RG * DL];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int D = a.D, Dp = padded8(D), R = a.H / a.G;
  int b = blockIdx.x;
  const int split = b % a.splits; b /= a.splits;
  const int hg = b % groups; b /= groups;
  const int g = b % a.G, r = b / a.G;
  const int i = a.pos[r], slot = a.slot[r];
  const int lo = i - a.window + 1 > 0 ? i - a.window + 1 : 0;
  const int per = (i - lo + a.splits) / a.splits;
  const int j0 = lo + split * per, j1 = j0 + per < i + 1 ? j0 + per : i + 1;
  const bool own = fused && j1 == i + 1 && j0 < j1;       // this part holds the row's own key

  const T* q = reinterpret_cast<const T*>(a.q) + (size_t)r * a.ld;
  const T* kp = reinterpret_cast<const T*>(a.k) + (size_t)r * a.ld;
  const int sub = lane % LPK, d0 = sub * 8, grp = wave * (64 / LPK) + lane / LPK;
  const int left = D - d0;               // elements of a row from d0 on
  const T* ring = reinterpret_cast<const T*>(a.ring) + ((size_t)slot * a.G + g) * a.ring_len * Dp;
  const float* rinv = a.rinv + (size_t)slot * a.ring_len;

  // a step's keys, as they lie in memory; the row's own key comes from the projection
  Raw8<T> kr[WR_KEYS];
  float ri[WR_KEYS];
  auto fetch = [&](int jb) {
#pragma unroll
    for (int u = 0; u < WR_KEYS; ++u) {
      const int j = jb + u * NG + grp;
      const int jc = j < j1 ? j : j1 - 1;
      const bool self = fused && jc == i;
      const int at = jc % a.ring_len;
      ri[u] = rinv[at];                                                   // (not used for the own key)
      const T* src = self ? kp + g * D + (left > 0 ? d0 : 0) : ring + (size_t)at * Dp + (left > 0 ? d0 : 0);
      kr[u].load(src, left > 0 && (!self || (vec && left >= 8)), left);
    }
  };
  // everything that does not depend on the sums below is requested before them
  if (j0 < j1) fetch(j0);
  float qv[RG][8], slope[RG];
  {
    float wk[8];
    load8(a.k_norm + g * D + (left > 0 ? d0 : 0), vec && left >= 8, left, wk);
#pragma unroll
    for (int h = 0; h < RG; ++h) {
      const int hr = hg * RG + h < R ? hg * RG + h : R - 1;              // a duplicate that is not stored
      const int head = g * R + hr;
      float wq[8];
      load8(q + head * D + (left > 0 ? d0 : 0), vec && left >= 8, left, qv[h]);
      load8(a.q_norm + head * D + (left > 0 ? d0 : 0), vec && left >= 8, left, wq);
      slope[h] = a.slopes[head];
#pragma unroll
      for (int e = 0; e < 8; ++e) qv[h][e] = qv[h][e] * wq[e] * (wk[e] * a.scale);
    }
  }
  float rq, rk = 0.f;
  if (fused) {
    const float qs = squares(q, a.H * D, vec), ks = own ? squares(kp, a.G * D, vec) : 0.f;
    rq = 1.0f / sqrtf(workgroup_sum<4>(qs, red[0]) / (float)(a.H * D) + a.eps);
    if (own) {
      rk = 1.0f / sqrtf(workgroup_sum<4>(ks, red[1]) / (float)(a.G * D) + a.eps);
      if (hg == 0) {
        put_ring_row(a, kp, g, slot, i);
        if (g == 0 && threadIdx.x == 0) a.rinv[(size_t)slot * a.ring_len + i % a.ring_len] = rk;
      }
    }
  } else {
    rq = a.q_scale[r];
  }

  float m[RG], l[RG], o[RG][8];
#pragma unroll
  for (int h = 0; h < RG; ++h) {
    m[h] = -1e30f;
    l[h] = 0.f;
#pragma unroll
    for (int e = 0; e < 8; ++e) o[h][e] = 0.f;
  }
  for (int jb = j0; jb < j1; jb += NG * WR_KEYS) {
    float kv[WR_KEYS][8], s[WR_KEYS][RG], rj[WR_KEYS];
    int dist[WR_KEYS];
#pragma unroll
    for (int u = 0; u < WR_KEYS; ++u) {
      const int j = jb + u * NG + grp;
      dist[u] = j < j1 ? i - j : -1;
      rj[u] = rq * (fused && dist[u] == 0 ? rk : ri[u]);
      kr[u].unpack(kv[u]);
    }
    if (jb + NG * WR_KEYS < j1) fetch(jb + NG * WR_KEYS);
#pragma unroll
    for (int h = 0; h < RG; ++h) {
      float top = m[h];
#pragma unroll
      for (int u = 0; u < WR_KEYS; ++u) {
        float t = 0.f;
#pragma unroll
        for (int e = 0; e < 8; ++e) t = __builtin_fmaf(qv[h][e], kv[u][e], t);
        t = group_sum<LPK>(t);
        s[u][h] = dist[u] >= 0 ? t * rj[u] - slope[h] * (float)dist[u] : -INFINITY;
        top = fmaxf(top, s[u][h]);
      }
      const float keep = exp_of<T>(m[h] - top);
      m[h] = top;
      l[h] *= keep;
#pragma unroll
      for (int e = 0; e < 8; ++e) o[h][e] *= keep;
#pragma unroll
      for (int u = 0; u < WR_KEYS; ++u) {
        const float p = exp_of<T>(s[u][h] - top);
        l[h] += p;
#pragma unroll
        for (int e = 0; e < 8; ++e) o[h][e] = __builtin_fmaf(p, kv[u][e], o[h][e]);
      }
    }
  }
#pragma unroll
  for (int h = 0; h < RG; ++h) {
    if (sub == 0) { sm[grp][h] = m[h]; sl[grp][h] = l[h]; }
    store8(so + (grp * RG + h) * DL + d0, o[h]);
  }
  __syncthreads();
  // the groups' states meet: sm becomes the weight of a group, red the total of a head
  __shared__ float top_s[RG], sum_s[RG];
  if (wave < RG) {                       // one wave per head (RG <= 4)
    const int h = wave;
    float mv = -1e30f, lv = 0.f;
    if (lane < NG) { mv = sm[lane][h]; lv = sl[lane][h]; }
    const float top = wave_max(mv);
    const float w = lane < NG ? exp_of<T>(mv - top) : 0.f;
    if (lane < NG) sm[lane][h] = w;
    const float tot = wave_sum(w * lv);
    if (lane == 0) { top_s[h] = top; sum_s[h] = tot; }
  }
  __syncthreads();
  for (int idx = threadIdx.x; idx < RG * D; idx += 256) {
    const int h = idx / D, d = idx % D;
    if (hg * RG + h >= R) continue;
    const int head = g * R + hg * RG + h;
    float t = 0.f;
#pragma unroll 4
    for (int n = 0; n < NG; ++n) t = __builtin_fmaf(sm[n][h], so[(n * RG + h) * DL + d], t);
    if (a.splits == 1) {
      const float gt = (float)(reinterpret_cast<const T*>(a.gate) + (size_t)r * a.ld)[head * D + d];
      (reinterpret_cast<T*>(a.out) + (size_t)r * a.out_ld)[head * D + d] = (T)(t / sum_s[h] * sigmoid_f32(gt));
    } else {
      part_o[(((size_t)r * a.H + head) * a.splits + split) * D + d] = t;
      if (d == 0) {
        float* ml = part_ml + (((size_t)r * a.H + head) * a.splits + split) * 2;
        ml[0] = top_s[h];
        ml[1] = sum_s[h];
      }
    }
  }
  if (a.splits == 1 && g == 0 && hg == 0)
    for (int c = a.H * D + threadIdx.x; c < a.out_ld; c += 256) (reinterpret_cast<T*>(a.out) + (size_t)r * a.out_ld)[c] = (T)0.0f;
}

// the parts of a row's window (at most 64) meet, and the gate is applied: one wave per (row, head)
template <typename T>
__global__ __launch_bounds__(64) void window_merge_kernel(WA a, const float* part_o, const float* part_ml) {
  __shared__ float weight[64];
  const int r = blockIdx.x / a.H, head = blockIdx.x % a.H, D = a.D, lane = threadIdx.x, n = a.splits;
  const size_t at = ((size_t)r * a.H + head) * n;
  const float* po = part_o + at * D;
  const T* gate = reinterpret_cast<const T*>(a.gate) + (size_t)r * a.ld + head * D;
  T* out = reinterpret_cast<T*>(a.out) + (size_t)r * a.out_ld;
  float m = -1e30f, l = 0.f;
  if (lane < n) { m = part_ml[(at + lane) * 2]; l = part_ml[(at + lane) * 2 + 1]; }
  // the first eight parts of this lane's first feature are requested before the weights are known
  float v[8];
#pragma unroll
  for (int u = 0; u < 8; ++u) v[u] = u < n && lane < D ? po[(size_t)u * D + lane] : 0.f;
  const float top = wave_max(m);
  const float w = lane < n ? exp_of<T>(m - top) : 0.f;
  weight[lane] = w;
  const float inv = 1.0f / wave_sum(w * l);
  __syncthreads();
  for (int d = lane; d < D; d += 64) {
    float t = 0.f;
    for (int s = 0; s < n; s += 8) {
      if (s > 0 || d != lane) {
#pragma unroll
        for (int u = 0; u < 8; ++u) v[u] = s + u < n ? po[(size_t)(s + u) * D + d] : 0.f;
      }
#pragma unroll
      for (int u = 0; u < 8; ++u) t = __builtin_fmaf(s + u < n ? weight[s + u] : 0.f, v[u], t);
    }
    out[head * D + d] = (T)(t * inv * sigmoid_f32((float)gate[d]));
  }
  if (head == 0)
    for (int c = a.H * D + lane; c < a.out_ld; c += 64) out[c] = (T)0.0f;
}

// ------------------------------------------------------------------------------------------
// Many rows on the matrix unit (bf16, D <= 32 * DT): a workgroup of four waves takes 64 * QW rows of one query head, a
// wave QW groups of 16; 64 keys at a time pass through LDS, once as they are (the A operand of S^T = K Q^T) and once
// transposed (the A operand of O^T = K^T P^T: the values are the keys).  A lane holds scores of ONE query, keys
// 16 t + 4 (lane / 16) + 0..3 of every 16-key group t; two groups are the eight values of a B operand as they stand if
// the transposed copy keeps its keys in that order: key 4 x + e of the first group of 32 goes to place 8 x + e, of the
// second to 8 x + 4 + e.
// ------------------------------------------------------------------------------------------
constexpr int WT_KEYS = 64;
constexpr int WT_VSTRIDE = WT_KEYS + 8;

template <int DT, int QW>
__global__ __launch_bounds__(256) void window_tile_kernel(WA a, bool vec) {
  constexpr int DM = DT * 32;
  constexpr int KS = DM + 8;
  constexpr int CH = DM / 8;                              // 16-byte pieces of a key row
  constexpr int ITEMS = WT_KEYS / 2 * CH;                 // (pair of keys, piece)
  constexpr int IPT = (ITEMS + 255) / 256;
  __shared__ __align__(16) bf16 sk[WT_KEYS * KS];
  __shared__ __align__(16) bf16 sv[DM * WT_VSTRIDE + DM];   // row d starts at d * WT_VSTRIDE + (d / 8) * 8
  __shared__ float sr[WT_KEYS];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, lg = lane >> 4, lc = lane & 15;
  const int head = blockIdx.x, tile = blockIdx.y;
  const int D = a.D, Dp = padded8(D), g = head / (a.H / a.G);
  const int skip = (int)blockIdx.z * 64 * QW;
  const int count = a.tile_count[tile] - skip;
  if (count <= 0) return;
  const int row0 = a.tile_row[tile] + skip;
  const int p0 = a.pos[row0], slot = a.slot[row0];
  const bf16* ring = reinterpret_cast<const bf16*>(a.ring) + ((size_t)slot * a.G + g) * a.ring_len * Dp;
  const float* rinv = a.rinv + (size_t)slot * a.ring_len;
  const float slope = a.slopes[head] * 1.4426950408889634f;

  // queries: lane holds features 32 m + 8 lg + 0..7 of row lc of each of its groups
  bf16x8 qf[QW][DT];
  int qi[QW];
#pragma unroll
  for (int w = 0; w < QW; ++w) {
    int n = (wave * QW + w) * 16 + lc;
    qi[w] = p0 + n;
    n = n < count ? n : count - 1;
    const bf16* q = reinterpret_cast<const bf16*>(a.q) + (size_t)(row0 + n) * a.ld + head * D;
    const float rq = a.q_scale[row0 + n] * a.scale * 1.4426950408889634f;
#pragma unroll
    for (int m = 0; m < DT; ++m) {
      const int d = m * 32 + lg * 8, left = D - d;
      float v[8], wq[8], wk[8];
      load8(q + (left > 0 ? d : 0), vec && left >= 8, left, v);
      load8(a.q_norm + head * D + (left > 0 ? d : 0), vec && left >= 8, left, wq);
      load8(a.k_norm + g * D + (left > 0 ? d : 0), vec && left >= 8, left, wk);
#pragma unroll
      for (int e = 0; e < 8; ++e) qf[w][m][e] = (bf16)(v[e] * rq * wq[e] * wk[e]);
    }
  }
  const int i_last = p0 + (count < 64 * QW ? count : 64 * QW) - 1;
  const int lo = p0 - a.window + 1 > 0 ? p0 - a.window + 1 : 0;
  const int w_first = p0 + wave * QW * 16, w_last = w_first + QW * 16 - 1;

  u32x4 pf[IPT][2];
  float pr = 0.f;
  auto fetch = [&](int jt) {
#pragma unroll
    for (int it = 0; it < IPT; ++it) {
      const int idx = threadIdx.x + it * 256, c = idx % CH, kp = idx / CH;
#pragma unroll
      for (int t = 0; t < 2; ++t) {
        const int j = jt + kp * 2 + t;
        pf[it][t] = u32x4{0, 0, 0, 0};
        if (idx < ITEMS && j <= i_last && c * 8 < Dp)
          pf[it][t] = *reinterpret_cast<const u32x4*>(ring + (size_t)(j % a.ring_len) * Dp + c * 8);
      }
    }
    if (threadIdx.x < WT_KEYS) {
      const int j = jt + threadIdx.x;
      pr = j <= i_last ? rinv[j % a.ring_len] : 0.f;
    }
  };
  auto stage = [&]() {
#pragma unroll
    for (int it = 0; it < IPT; ++it) {
      const int idx = threadIdx.x + it * 256, c = idx % CH, kp = idx / CH;
      if (idx >= ITEMS) break;
      *reinterpret_cast<u32x4*>(sk + (kp * 2) * KS + c * 8) = pf[it][0];
      *reinterpret_cast<u32x4*>(sk + (kp * 2 + 1) * KS + c * 8) = pf[it][1];
      const int k32 = (kp * 2) & 31, place = ((kp * 2) & 32) + ((k32 & 15) >> 2) * 8 + (k32 >> 4) * 4 + (k32 & 3);
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const uint32_t x = pf[it][0][e], y = pf[it][1][e];
        bf16* base = sv + (c * 8 + 2 * e) * WT_VSTRIDE + c * 8 + place;
        *reinterpret_cast<uint32_t*>(base) = (x & 0xffffu) | (y << 16);
        *reinterpret_cast<uint32_t*>(base + WT_VSTRIDE) = (x >> 16) | (y & 0xffff0000u);
      }
    }
    if (threadIdx.x < WT_KEYS) sr[threadIdx.x] = pr;
  };

  f32x4 o[QW][DT * 2];
  float m[QW], l[QW];
#pragma unroll
  for (int w = 0; w < QW; ++w) {
    m[w] = -1e30f;
    l[w] = 0.f;
#pragma unroll
    for (int t = 0; t < DT * 2; ++t) o[w][t] = f32x4{0.f, 0.f, 0.f, 0.f};
  }
  const int j_begin = lo / WT_KEYS * WT_KEYS;
  fetch(j_begin);
  for (int jt = j_begin; jt <= i_last; jt += WT_KEYS) {
    __syncthreads();
    stage();
    __syncthreads();
    if (jt + WT_KEYS <= i_last) fetch(jt + WT_KEYS);
    if (jt > w_last || jt + WT_KEYS - 1 < w_first - a.window + 1) continue;       // nothing this wave's rows see
    f32x4 s[QW][4];
#pragma unroll
    for (int t = 0; t < 4; ++t) {
#pragma unroll
      for (int w = 0; w < QW; ++w) s[w][t] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int c = 0; c < DT; ++c) {
        const bf16x8 kf = *reinterpret_cast<const bf16x8*>(sk + (t * 16 + lc) * KS + c * 32 + lg * 8);
#pragma unroll
        for (int w = 0; w < QW; ++w) s[w][t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf, qf[w][c], s[w][t], 0, 0, 0);
      }
    }
    bf16x8 p[QW][2];
#pragma unroll
    for (int w = 0; w < QW; ++w) {
      float top = m[w];
#pragma unroll
      for (int t = 0; t < 4; ++t) {
        const f32x4 ri = *reinterpret_cast<const f32x4*>(sr + t * 16 + lg * 4);
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          const int dist = qi[w] - (jt + t * 16 + lg * 4 + e);
          const float v = s[w][t][e] * ri[e] - slope * (float)dist;
          s[w][t][e] = dist >= 0 && dist < a.window ? v : -INFINITY;
          top = fmaxf(top, s[w][t][e]);
        }
      }
      top = fmaxf(top, __shfl_xor(top, 16, 64));
      top = fmaxf(top, __shfl_xor(top, 32, 64));
      const float keep = exp2f(m[w] - top);
      m[w] = top;
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
      for (int t = 0; t < DT * 2; ++t)
#pragma unroll
        for (int e = 0; e < 4; ++e) o[w][t][e] *= keep;
    }
#pragma unroll
    for (int t = 0; t < DT * 2; ++t)
#pragma unroll
      for (int kg = 0; kg < 2; ++kg) {
        const int d = t * 16 + lc;
        const bf16x8 vf = *reinterpret_cast<const bf16x8*>(sv + d * WT_VSTRIDE + (d >> 3) * 8 + kg * 32 + lg * 8);
#pragma unroll
        for (int w = 0; w < QW; ++w) o[w][t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf, p[w][kg], o[w][t], 0, 0, 0);
      }
  }
#pragma unroll
  for (int w = 0; w < QW; ++w) {
    float tot = l[w];
    tot += __shfl_xor(tot, 16, 64);
    tot += __shfl_xor(tot, 32, 64);
    const int n = (wave * QW + w) * 16 + lc;
    if (n >= count) continue;
    const bf16* gate = reinterpret_cast<const bf16*>(a.gate) + (size_t)(row0 + n) * a.ld + head * D;
    bf16* out = reinterpret_cast<bf16*>(a.out) + (size_t)(row0 + n) * a.out_ld + head * D;
    const float inv = 1.0f / tot;
#pragma unroll
    for (int t = 0; t < DT * 2; ++t) {
      const int d = t * 16 + lg * 4;
      if (vec && d + 4 <= D) {
        const bf16x4 gv = *reinterpret_cast<const bf16x4*>(gate + d);
        bf16x4 y;
#pragma unroll
        for (int e = 0; e < 4; ++e) y[e] = (bf16)(o[w][t][e] * inv / (1.0f + __expf(-(float)gv[e])));
        *reinterpret_cast<bf16x4*>(out + d) = y;
      } else {
#pragma unroll
        for (int e = 0; e < 4; ++e)
          if (d + e < D) out[d + e] = (bf16)(o[w][t][e] * inv / (1.0f + __expf(-(float)gate[d + e])));
      }
    }
    if (head == 0 && lg == 0)
      for (int c = a.H * D; c < a.out_ld; ++c) (reinterpret_cast<bf16*>(a.out) + (size_t)(row0 + n) * a.out_ld)[c] = (bf16)0.0f;
  }
}

// ------------------------------------------------------------------------------------------
static int check_window(const WA& a, const char* name) {
  PTA_REQUIRE(a.dtype == PTA_BF16 || a.dtype == PTA_FP32, "%s: unknown type %d", name, a.dtype);
  PTA_REQUIRE(a.rows > 0 && a.H > 0 && a.G > 0 && a.H % a.G == 0, "%s: rows %d, heads %d, key heads %d", name, a.rows, a.H, a.G);
  PTA_REQUIRE(a.D > 0 && a.D <= 512, "%s: head size %d (1 .. 512)", name, a.D);
  PTA_REQUIRE(a.q && a.k && a.gate && a.q_norm && a.k_norm && a.slopes && a.ring && a.rinv && a.slot && a.pos,
              "%s: null pointer", name);
  PTA_REQUIRE(a.window > 0 && a.ring_len > 0, "%s: window %d, ring of %d", name, a.window, a.ring_len);
  PTA_REQUIRE(a.ld >= a.H * a.D && pta_aligned(a.ring, 16), "%s: row stride %d, or the ring's alignment", name, a.ld);
  return PTA_OK;
}

// whole 16-byte pieces everywhere a head's features are read from the projection rows
static bool vectors_fit(const WA& a) {
  const size_t es = a.dtype == PTA_BF16 ? 2 : 4;
  return a.D % 8 == 0 && (size_t)a.ld * es % 16 == 0 && pta_aligned(a.q, 16) && pta_aligned(a.k, 16) && pta_aligned(a.gate, 16) &&
         (size_t)a.out_ld * es % 8 == 0 && pta_aligned(a.out, 8) && pta_aligned(a.q_norm, 16) && pta_aligned(a.k_norm, 16);
}

template <typename T, int RG>
static void launch_rows_for(const WA& a, int fused, float* po, float* pml, hipStream_t s) {
  const int groups = (a.H / a.G + RG - 1) / RG;
  const dim3 grid((unsigned)((size_t)a.rows * a.G * groups * a.splits));
  const bool vec = vectors_fit(a);
  if (a.D <= 32) hipLaunchKernelGGL((window_rows_kernel<T, RG, 4>), grid, dim3(256), 0, s, a, vec, fused, groups, po, pml);
  else if (a.D <= 64) hipLaunchKernelGGL((window_rows_kernel<T, RG, 8>), grid, dim3(256), 0, s, a, vec, fused, groups, po, pml);
  else if (a.D <= 128) hipLaunchKernelGGL((window_rows_kernel<T, RG, 16>), grid, dim3(256), 0, s, a, vec, fused, groups, po, pml);
  else if (a.D <= 256) hipLaunchKernelGGL((window_rows_kernel<T, RG, 32>), grid, dim3(256), 0, s, a, vec, fused, groups, po, pml);
  else hipLaunchKernelGGL((window_rows_kernel<T, RG, 64>), grid, dim3(256), 0, s, a, vec, fused, groups, po, pml);
}

template <typename T>
static void launch_rows(const WA& a, int fused, float* po, float* pml, hipStream_t s) {
  const int R = a.H / a.G;
  if (R == 1) launch_rows_for<T, 1>(a, fused, po, pml, s);
  else if (R == 2) launch_rows_for<T, 2>(a, fused, po, pml, s);
  else launch_rows_for<T, 4>(a, fused, po, pml, s);
}

extern "C" int pta_window_append(const WA* args, pta_stream_t stream) {
  PTA_REQUIRE(args, "pta_window_append: null arguments");
  const WA& a = *args;
  const int rc = check_window(a, "pta_window_append");
  if (rc) return rc;
  PTA_REQUIRE(a.q_scale, "pta_window_append: q_scale is missing");
  if (a.dtype == PTA_BF16) hipLaunchKernelGGL((window_append_kernel<bf16>), dim3(a.rows), dim3(256), 0, (hipStream_t)stream, a, vectors_fit(a));
  else hipLaunchKernelGGL((window_append_kernel<float>), dim3(a.rows), dim3(256), 0, (hipStream_t)stream, a, vectors_fit(a));
  PTA_CHECK_LAUNCH("pta_window_append");
  return PTA_OK;
}

extern "C" int pta_window_attention(const WA* args, pta_stream_t stream) {
  PTA_REQUIRE(args, "pta_window_attention: null arguments");
  WA a = *args;
  const int rc = check_window(a, "pta_window_attention");
  if (rc) return rc;
  PTA_REQUIRE(a.q_scale && a.out && a.out_ld >= a.H * a.D, "pta_window_attention: q_scale or the output is missing");
  hipStream_t s = (hipStream_t)stream;
  a.splits = 1;
  if (a.dtype == PTA_FP32 || a.D > 256) {
    if (a.dtype == PTA_FP32) launch_rows<float>(a, 0, nullptr, nullptr, s);
    else launch_rows<bf16>(a, 0, nullptr, nullptr, s);
  } else {
    PTA_REQUIRE(a.tiles > 0 && a.tile_row && a.tile_count, "pta_window_attention: the rows' tiles are missing");
    PTA_REQUIRE(a.tiles <= 65535, "pta_window_attention: %d tiles (at most 65535)", a.tiles);
    const bool vec = vectors_fit(a);
    const dim3 one(a.H, a.tiles, 1), two(a.H, a.tiles, 2);
    if (a.D <= 32) hipLaunchKernelGGL((window_tile_kernel<1, 2>), one, dim3(256), 0, s, a, vec);
    else if (a.D <= 64) hipLaunchKernelGGL((window_tile_kernel<2, 2>), one, dim3(256), 0, s, a, vec);
    else if (a.D <= 96) hipLaunchKernelGGL((window_tile_kernel<3, 2>), one, dim3(256), 0, s, a, vec);
    else if (a.D <= 128) hipLaunchKernelGGL((window_tile_kernel<4, 2>), one, dim3(256), 0, s, a, vec);
    else hipLaunchKernelGGL((window_tile_kernel<8, 1>), two, dim3(256), 0, s, a, vec);
  }
  PTA_CHECK_LAUNCH("pta_window_attention");
  return PTA_OK;
}

extern "C" size_t pta_window_attention_workspace_bytes(int rows, int H, int D, int splits) {
  if (rows <= 0 || H <= 0 || D <= 0 || splits <= 1) return 0;
  return (size_t)rows * H * splits * (D + 2) * sizeof(float);
}

extern "C" int pta_window_decode(const WA* args, pta_stream_t stream) {
  PTA_REQUIRE(args, "pta_window_decode: null arguments");
  const WA& a = *args;
  const int rc = check_window(a, "pta_window_decode");
  if (rc) return rc;
  PTA_REQUIRE(a.out && a.out_ld >= a.H * a.D && a.splits >= 1 && a.splits <= 64, "pta_window_decode: output, or splits %d (1 .. 64)", a.splits);
  const size_t need = pta_window_attention_workspace_bytes(a.rows, a.H, a.D, a.splits);
  PTA_REQUIRE(a.splits == 1 || (a.workspace && a.workspace_bytes >= need), "pta_window_decode: the workspace needs %zu bytes", need);
  hipStream_t s = (hipStream_t)stream;
  float* po = (float*)a.workspace;
  float* pml = po ? po + (size_t)a.rows * a.H * a.splits * a.D : nullptr;
  if (a.dtype == PTA_BF16) launch_rows<bf16>(a, 1, po, pml, s);
  else launch_rows<float>(a, 1, po, pml, s);
  if (a.splits > 1) {
    if (a.dtype == PTA_BF16) hipLaunchKernelGGL((window_merge_kernel<bf16>), dim3(a.rows * a.H), dim3(64), 0, s, a, po, pml);
    else hipLaunchKernelGGL((window_merge_kernel<float>), dim3(a.rows * a.H), dim3(64), 0, s, a, po, pml);
  }
  PTA_CHECK_LAUNCH("pta_window_decode");
  return PTA_OK;
}
