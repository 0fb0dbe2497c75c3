// Attention over cached keys and values with norms per head, rotation, windows that keep the first positions, chunks, sinks,
// differential pairs of maps, output gates, penalties of the distance and short convolutions ahead of it all.
//
// The keys a row sees are numbered: first the kept positions, then those from the window's (or chunk's) begin on.  Every kernel
// works on a stretch of these numbers, so positions nobody sees cost nothing.
#include "short_conv.h"

typedef pta_head_attention_args HA;

constexpr float LOG2E = 1.4426950408889634f;

__device__ __forceinline__ int first_visible(const HA& a, int i) {
  const int lo = i - a.window + 1 > 0 ? i - a.window + 1 : 0;
  const int begin = a.chunk ? i / a.chunk * a.chunk : 0;
  return lo > begin ? lo : begin;
}

// numbers -> positions and cache rows, for rows that see nothing between `keep` and lo
struct KeyRange {
  int kept, lo, at, ring, keep;
  __device__ __forceinline__ KeyRange(const HA& a, int first) {
    lo = first;
    keep = a.keep;
    ring = a.ring_len - keep;
    kept = lo <= keep ? 1 << 30 : keep;                   // no gap: numbers are positions, and rows
    at = lo <= keep ? 0 : (int)((unsigned)(lo - keep) % (unsigned)ring);
  }
  __device__ __forceinline__ int count(int last) const { return lo <= keep ? last + 1 : keep + last - lo + 1; }
  __device__ __forceinline__ int position(int n) const { return n < kept ? n : lo + n - kept; }
  __device__ __forceinline__ int row(int n) const {
    if (n < kept) return n;
    const int r = at + n - kept;
    return keep + (r >= ring ? r - ring : r);
  }
};

__device__ __forceinline__ int ring_row(const HA& a, int p) {
  return p < a.keep ? p : a.keep + (int)((unsigned)(p - a.keep) % (unsigned)(a.ring_len - a.keep));
}
// what a distance takes off a score of head h
template <typename T> __device__ __forceinline__ float log_of(float x);
template <> __device__ __forceinline__ float log_of<float>(float x) { return logf(x); }
template <> __device__ __forceinline__ float log_of<bf16>(float x) { return __logf(x); }

__device__ __forceinline__ const float* angles_of(const HA& a, int pos) {
  return a.cos_sin + (size_t)(pos < a.positions ? pos : a.positions - 1) * a.rot;
}

// Eight features of a head from d0 on, LPK lanes holding a head (zeros past D): norm, then rotation by cs (a row of cos_sin).
template <int LPK>
__device__ __forceinline__ void norm_rotate(const HA& a, const float (&w)[8], bool normed, int d0, const float* cs, float (&v)[8]) {
  if (normed) {
    float s = 0.f;
#pragma unroll
    for (int e = 0; e < 8; ++e) s = __builtin_fmaf(v[e], v[e], s);
    const float inv = 1.0f / sqrtf(group_sum<LPK>(s) / (float)a.dim + a.eps);
#pragma unroll
    for (int e = 0; e < 8; ++e) v[e] = v[e] * inv * w[e];
  }
  if (d0 < a.rot) rotate8(cs + d0, v);
}

// ------------------------------------------------------------------------------------------
// Keys and values of a row into the cache
// ------------------------------------------------------------------------------------------
template <typename T, int LPK>
__global__ __launch_bounds__(256) void head_append_kernel(HA a) {
  constexpr int NG = 256 / LPK;
  const int r = blockIdx.x, pos = a.pos[r], slot = a.slot[r];
  const int sub = threadIdx.x % LPK, grp = threadIdx.x / LPK, d0 = sub * 8;
  const int nk = a.G * a.maps, row = ring_row(a, pos);
  const bool in = d0 < a.D;
  float w[8];
  load8(a.k_norm ? a.k_norm + (in ? d0 : 0) : nullptr, a.k_norm != nullptr, 0, w);
  for (int j0 = 0; j0 < nk; j0 += NG) {                   // (the same turns for all: the sums run over whole lane groups)
    const int j = j0 + grp < nk ? j0 + grp : nk - 1;
    float v[8];
    load8(reinterpret_cast<const T*>(a.k) + (size_t)r * a.ld + j * a.D + (in ? d0 : 0), in, 0, v);
    if (!in)
#pragma unroll
      for (int e = 0; e < 8; ++e) v[e] = 0.f;
    norm_rotate<LPK>(a, w, a.k_norm != nullptr, d0, angles_of(a, pos), v);
    if (in && j0 + grp < nk) store8(reinterpret_cast<T*>(a.keys) + (((size_t)slot * nk + j) * a.ring_len + row) * a.D + d0, v);
  }
  for (int c = threadIdx.x; c < a.G * a.E / 8; c += 256) {
    const int g = c / (a.E / 8), d = c % (a.E / 8) * 8;
    float v[8];
    load8(reinterpret_cast<const T*>(a.v) + (size_t)r * a.ld + g * a.E + d, true, 8, v);
    store8(reinterpret_cast<T*>(a.values) + (((size_t)slot * a.G + g) * a.ring_len + row) * a.E + d, v);
  }
}

// ------------------------------------------------------------------------------------------
// The end of a head: value(t, d) is feature d of map t's weighted sum, inv[t] one over its denominator.  One wave.
// ------------------------------------------------------------------------------------------
template <typename T, int MAPS, class Value>
__device__ __forceinline__ void finish_head(const HA& a, int r, int head, int lane, const float (&inv)[MAPS], Value value) {
  T* out = reinterpret_cast<T*>(a.out) + ((size_t)r * a.H + head) * a.E;
  const T* gate = a.gate ? reinterpret_cast<const T*>(a.gate) + (size_t)r * a.ld + head * a.E : nullptr;
  const float hg = a.head_gate ? sigmoid_f32(a.head_gate[(size_t)r * a.H + head]) : 1.0f;
  float f = hg;
  auto combined = [&](int d) {
    if constexpr (MAPS == 2) return value(0, d) * inv[0] - a.lambda * (value(1, d) * inv[1]);
    else return value(0, d) * inv[0];
  };
  if constexpr (MAPS == 2) {
    float s = 0.f;
    for (int d = lane; d < a.E; d += 64) {
      const float o = combined(d);
      s = __builtin_fmaf(o, o, s);
    }
    f *= (1.0f - a.diff) / sqrtf(wave_sum(s) / (float)a.vdim + a.eps);
  }
  for (int d = lane; d < a.E; d += 64) {
    float o = combined(d) * f;
    if (gate) o *= sigmoid_f32((float)gate[d]);
    out[d] = (T)o;
  }
}

// ------------------------------------------------------------------------------------------
// Row by row on the vector unit: a workgroup per (row, key head, RG of its query heads, part of the visible keys).  LPK lanes
// share a key (eight features each) and its value, for the RG heads and the maps.  `fused`: the row's own key and value come
// from the projection and are put into the cache by this launch.  FAR: there may be a penalty of the distance, or convolutions.
// ------------------------------------------------------------------------------------------
constexpr int HR_KEYS = 4;               // keys a lane group takes per step

template <typename T, int RG, int MAPS, int LPK, bool FAR>
__global__ __launch_bounds__(256) void head_rows_kernel(HA a, int fused, int groups, float* part_o, float* part_ml) {
  constexpr int NG = 256 / LPK, DL = LPK * 8, NQ = RG * MAPS;
  __shared__ float sm[NG][NQ], sl[NG][NQ], inv_s[NQ];
  __shared__ __align__(16) float so[NG * NQ * DL];
  __shared__ float res[NQ * DL];
  __shared__ __align__(16) float s_conv[FAR ? (RG + 2) * DL : 8];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int D = a.D, E = a.E, R = a.H / a.G;
  int b = blockIdx.x;
  const int split = b % a.splits; b /= a.splits;
  const int hg = b % groups; b /= groups;
  const int g = b % a.G, r = b / a.G;
  const int i = a.pos[r], slot = a.slot[r];
  const KeyRange keys(a, first_visible(a, i));
  const int total = keys.count(i), per = (total + a.splits - 1) / a.splits;
  const int n0 = split * per, n1 = n0 + per < total ? n0 + per : total;
  const bool own = fused && n1 == total && n0 < n1;       // this part holds the row's own key
  const int n_end = own ? n1 - 1 : n1;                    // numbers that are read from the cache

  const int sub = lane % LPK, d0 = sub * 8, grp = wave * (64 / LPK) + lane / LPK;
  const bool dk = d0 < D, dv = d0 < E;
  const T* kring = reinterpret_cast<const T*>(a.keys) + (((size_t)slot * a.G + g) * MAPS * a.ring_len) * D + (dk ? d0 : 0);
  const T* vring = reinterpret_cast<const T*>(a.values) + (((size_t)slot * a.G + g) * a.ring_len) * E + (dv ? d0 : 0);

  Raw8<T> kr[HR_KEYS][MAPS], vr[HR_KEYS];
  auto fetch = [&](int nb) {
#pragma unroll
    for (int u = 0; u < HR_KEYS; ++u) {
      const int n = nb + u * NG + grp, row = keys.row(n < n_end ? n : n_end - 1);
#pragma unroll
      for (int t = 0; t < MAPS; ++t) kr[u][t].load(kring + ((size_t)t * a.ring_len + row) * D, true, 8);
      vr[u].load(vring + (size_t)row * E, true, 8);
    }
  };
  if (n0 < n_end) fetch(n0);               // (before everything that does not depend on it)

  const T* proj_q = reinterpret_cast<const T*>(a.q) + (size_t)r * a.ld;
  const float* cs = a.rot ? angles_of(a, i) : nullptr;
  auto zero_past = [&](bool in, float (&v)[8]) {
    if (!in)
#pragma unroll
      for (int e = 0; e < 8; ++e) v[e] = 0.f;
  };
  float qv[NQ][8], wn[8], far1[RG], far2[RG];
  load8(a.q_norm ? a.q_norm + (dk ? d0 : 0) : nullptr, a.q_norm != nullptr, 0, wn);
#pragma unroll
  for (int h = 0; h < RG; ++h) {
    const int head = g * R + (hg * RG + h < R ? hg * RG + h : R - 1);               // (a duplicate that is not stored)
#pragma unroll
    for (int t = 0; t < MAPS; ++t) load8(proj_q + (head * MAPS + t) * D + (dk ? d0 : 0), true, 8, qv[h * MAPS + t]);
    far1[h] = FAR && a.far1 ? a.far1[head] : 0.f;
    far2[h] = FAR && a.far1 ? a.far2[head] : 0.f;
  }
  const bool convolved = FAR && fused && a.conv.ring;
  if constexpr (FAR) {
    if (convolved) {                                      // the workgroup's queries, and the row's own key and value: a thread per piece
      for (int p = threadIdx.x; p < (RG + 2) * LPK; p += 256) {
        const int which = p / LPK, d = p % LPK * 8;
        if (d >= (which <= RG ? D : E) || (which >= RG && !own)) continue;
        const int hr = hg * RG + which < R ? hg * RG + which : R - 1;
        const int c0 = (which < RG ? (g * R + hr) * D : which == RG ? (a.H + g) * D : (a.H + a.G) * D + g * E) + d;
        float v[8];
        load8(proj_q + c0, true, 8, v);
        if (which < RG ? split == 0 && hg * RG + which < R : hg == 0) store8(conv_place<T>(a.conv, slot, i, c0), v);
        conv8<T>(a.conv, slot, i, c0, v);
        store8(s_conv + p * 8, v);
      }
      __syncthreads();
#pragma unroll
      for (int h = 0; h < RG; ++h) load8(s_conv + (h * LPK + sub) * 8, true, 8, qv[h]);
    }
  }
#pragma unroll
  for (int q = 0; q < NQ; ++q) {
    zero_past(dk, qv[q]);
    norm_rotate<LPK>(a, wn, a.q_norm != nullptr, d0, cs, qv[q]);
#pragma unroll
    for (int e = 0; e < 8; ++e) qv[q][e] *= a.scale;
  }

  float m[NQ], l[NQ], o[NQ][8];
#pragma unroll
  for (int q = 0; q < NQ; ++q) {
    m[q] = -1e30f;
    l[q] = 0.f;
#pragma unroll
    for (int e = 0; e < 8; ++e) o[q][e] = 0.f;
  }
  // U keys of this lane group, those with `seen`, `back` positions before the row
  auto step = [&](auto count, const auto& kv, const auto& vv, const auto& seen, const auto& back) {
    constexpr int U = decltype(count)::value;
#pragma unroll
    for (int q = 0; q < NQ; ++q) {
      float s[U], top = m[q];
#pragma unroll
      for (int u = 0; u < U; ++u) {
        float t = 0.f;
#pragma unroll
        for (int e = 0; e < 8; ++e) t = __builtin_fmaf(qv[q][e], kv[u][q % MAPS][e], t);
        t = group_sum<LPK>(t);
        if constexpr (FAR) t -= far1[q / MAPS] * log_of<T>(1.0f + far2[q / MAPS] * back[u]);
        s[u] = seen[u] ? t : -INFINITY;
        top = fmaxf(top, s[u]);
      }
      const float keep = exp_of<T>(m[q] - top);
      m[q] = top;
      l[q] *= keep;
#pragma unroll
      for (int e = 0; e < 8; ++e) o[q][e] *= keep;
#pragma unroll
      for (int u = 0; u < U; ++u) {
        const float p = exp_of<T>(s[u] - top);
        l[q] += p;
#pragma unroll
        for (int e = 0; e < 8; ++e) o[q][e] = __builtin_fmaf(p, vv[u][e], o[q][e]);
      }
    }
  };
  for (int nb = n0; nb < n_end; nb += NG * HR_KEYS) {
    float kv[HR_KEYS][MAPS][8], vv[HR_KEYS][8];
    bool seen[HR_KEYS];
    float back[HR_KEYS];
#pragma unroll
    for (int u = 0; u < HR_KEYS; ++u) {
      const int n = nb + u * NG + grp;
      seen[u] = n < n_end;
      back[u] = FAR && seen[u] ? (float)(i - keys.position(n)) : 0.f;
#pragma unroll
      for (int t = 0; t < MAPS; ++t) kr[u][t].unpack(kv[u][t]);
      vr[u].unpack(vv[u]);
    }
    if (nb + NG * HR_KEYS < n_end) fetch(nb + NG * HR_KEYS);
    step(std::integral_constant<int, HR_KEYS>{}, kv, vv, seen, back);
  }
  if (own) {
    float kv[1][MAPS][8], vv[1][8];
    load8(a.k_norm ? a.k_norm + (dk ? d0 : 0) : nullptr, a.k_norm != nullptr, 0, wn);
    const T* pk = reinterpret_cast<const T*>(a.k) + (size_t)r * a.ld + g * MAPS * D + (dk ? d0 : 0);
    load8(reinterpret_cast<const T*>(a.v) + (size_t)r * a.ld + g * E + (dv ? d0 : 0), true, 8, vv[0]);
    const bool put = hg == 0 && grp == 0;
    const int row = ring_row(a, i);
    if (convolved) {
      load8(s_conv + ((RG + 1) * LPK + sub) * 8, true, 8, vv[0]);
      zero_past(dv, vv[0]);
    }
#pragma unroll
    for (int t = 0; t < MAPS; ++t) {
      load8(pk + t * D, true, 8, kv[0][t]);
      if (convolved) load8(s_conv + (RG * LPK + sub) * 8, true, 8, kv[0][t]);
      zero_past(dk, kv[0][t]);
      norm_rotate<LPK>(a, wn, a.k_norm != nullptr, d0, cs, kv[0][t]);
      if (put && dk) store8(const_cast<T*>(kring) + ((size_t)t * a.ring_len + row) * D, kv[0][t]);
#pragma unroll
      for (int e = 0; e < 8; ++e) kv[0][t][e] = (float)(T)kv[0][t][e];                // what the cache holds
    }
    if (put && dv) store8(const_cast<T*>(vring) + (size_t)row * E, vv[0]);
    const bool seen[1] = {grp == 0};
    const float back[1] = {0.f};
    step(std::integral_constant<int, 1>{}, kv, vv, seen, back);
  }
#pragma unroll
  for (int q = 0; q < NQ; ++q) {
    if (sub == 0) { sm[grp][q] = m[q]; sl[grp][q] = l[q]; }
    store8(so + (grp * NQ + q) * DL + d0, o[q]);
  }
  __syncthreads();
  // the groups' states meet: sm becomes the weight of a group
  if (wave < NQ) {                       // one wave per head and map (NQ <= 4)
    const int q = wave, hr = hg * RG + q / MAPS;
    float mv = -1e30f, lv = 0.f;
    if (lane < NG) { mv = sm[lane][q]; lv = sl[lane][q]; }
    float top = wave_max(mv), sink = 0.f;
    if (a.sink && split == 0 && hr < R) {
      const float z = a.sink[g * R + hr];
      top = fmaxf(top, z);
      sink = exp_of<T>(z - top);
    }
    const float w = lane < NG ? exp_of<T>(mv - top) : 0.f;
    if (lane < NG) sm[lane][q] = w;
    const float tot = wave_sum(w * lv) + sink;
    if (lane == 0) {
      inv_s[q] = 1.0f / tot;
      if (a.splits > 1 && hr < R) {
        float* ml = part_ml + ((((size_t)r * a.H + g * R + hr) * MAPS + q % MAPS) * a.splits + split) * 2;
        ml[0] = top;
        ml[1] = tot;
      }
    }
  }
  __syncthreads();
  for (int idx = threadIdx.x; idx < NQ * E; idx += 256) {
    const int q = idx / E, d = idx % E, hr = hg * RG + q / MAPS;
    float t = 0.f;
#pragma unroll 4
    for (int n = 0; n < NG; ++n) t = __builtin_fmaf(sm[n][q], so[(n * NQ + q) * DL + d], t);
    if (a.splits == 1) res[q * DL + d] = t;
    else if (hr < R) part_o[((((size_t)r * a.H + g * R + hr) * MAPS + q % MAPS) * a.splits + split) * E + d] = t;
  }
  if (a.splits > 1) return;
  __syncthreads();
  if (wave < RG && hg * RG + wave < R) {
    float inv[MAPS];
#pragma unroll
    for (int t = 0; t < MAPS; ++t) inv[t] = inv_s[wave * MAPS + t];
    finish_head<T, MAPS>(a, r, g * R + hg * RG + wave, lane, inv, [&](int t, int d) { return res[(wave * MAPS + t) * DL + d]; });
  }
}

// the parts of a row's keys (at most 64) meet: one workgroup per (row, head), a thread per map and feature
template <typename T, int MAPS>
__global__ __launch_bounds__(256) void head_merge_kernel(HA a, const float* part_o, const float* part_ml) {
  __shared__ float weight[MAPS][64], inv_s[MAPS];
  __shared__ float res[MAPS * 512];
  const int r = blockIdx.x / a.H, head = blockIdx.x % a.H, E = a.E, lane = threadIdx.x & 63, wave = threadIdx.x >> 6, n = a.splits;
  const size_t at = ((size_t)r * a.H + head) * MAPS * n;
  // the first eight parts of this thread's first feature are requested before the weights are known
  auto fetch = [&](int i, int s, float (&v)[8]) {
    const int t = i / E, d = i % E;
#pragma unroll
    for (int u = 0; u < 8; ++u) v[u] = i < MAPS * E && s + u < n ? part_o[(at + t * n + s + u) * E + d] : 0.f;
  };
  float v[8];
  fetch(threadIdx.x, 0, v);
  if (wave < MAPS) {
    float m = -1e30f, l = 0.f;
    if (lane < n) { m = part_ml[(at + wave * n + lane) * 2]; l = part_ml[(at + wave * n + lane) * 2 + 1]; }
    const float top = wave_max(m), w = lane < n ? exp_of<T>(m - top) : 0.f;
    weight[wave][lane] = w;
    const float total = wave_sum(w * l);
    if (lane == 0) inv_s[wave] = 1.0f / total;
  }
  __syncthreads();
  for (int i = threadIdx.x; i < MAPS * E; i += 256) {
    float sum = 0.f;
    for (int s = 0; s < n; s += 8) {
      float next[8];
      if (s + 8 < n) fetch(i, s + 8, next);
      else fetch(i + 256, 0, next);
#pragma unroll
      for (int u = 0; u < 8; ++u) sum = __builtin_fmaf(s + u < n ? weight[i / E][s + u] : 0.f, v[u], sum);
#pragma unroll
      for (int u = 0; u < 8; ++u) v[u] = next[u];
    }
    res[i] = sum;
  }
  __syncthreads();
  if (wave > 0) return;
  float inv[MAPS];
#pragma unroll
  for (int t = 0; t < MAPS; ++t) inv[t] = inv_s[t];
  finish_head<T, MAPS>(a, r, head, lane, inv, [&](int t, int d) { return res[t * E + d]; });
}

// ------------------------------------------------------------------------------------------
// Many rows on the matrix unit (bf16, D and E up to 256): a workgroup of four waves takes 128 rows of one head, a wave 2 groups
// of 16 queries - of two maps: 64 rows, the groups being the two maps of the same 16 rows, so that the values are read once.
// 64 keys at a time pass through LDS.  S^T = K Q^T, O^T = V^T P^T.  A lane holds scores of ONE query, keys 16 t + 4 (lane / 16) +
// 0..3 of every 16-key group t; two groups are the eight values of a B operand as they stand, and the transposed reads of V take
// the keys in that order.
// ------------------------------------------------------------------------------------------
constexpr int HT_KEYS = 64;

template <int DKT, int DVT, int MAPS>
constexpr size_t head_tile_smem() { return (size_t)HT_KEYS * (MAPS * (DKT * 32 + 8) + (DVT + 1) / 2 * 32 + 8) * sizeof(bf16); }

template <int DKT, int DVT, int MAPS>
__global__ __launch_bounds__(256) void head_tile_kernel(HA a) {
  constexpr int QW = 2, RW = QW / MAPS * 16, KS = DKT * 32 + 8, VIT = (DVT + 1) / 2, VS = VIT * 32 + 8;
  extern __shared__ __align__(16) unsigned char head_tile_lds[];
  bf16* sk = reinterpret_cast<bf16*>(head_tile_lds);                   // [MAPS][HT_KEYS][KS]
  bf16* sv = sk + MAPS * HT_KEYS * KS;                                 // [HT_KEYS][VS]
  // of the distance from row n of the workgroup's to key k of a step, at k - n + (rows - 1): what is taken off the score
  __shared__ float far[HT_KEYS + 4 * RW];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, lg = lane >> 4, lc = lane & 15;
  const int head = blockIdx.x, tile = blockIdx.y, skip = (int)blockIdx.z * 4 * RW;
  const int D = a.D, E = a.E, g = head / (a.H / a.G);
  int count = a.tile_count[tile] - skip;
  if (count <= 0) return;
  count = count < 4 * RW ? count : 4 * RW;
  const int row0 = a.tile_row[tile] + skip, p0 = a.pos[row0], slot = a.slot[row0];

  // queries: lane holds features 32 m + 8 lg + 0..7 of row lc of each of its groups
  bf16x8 qf[QW][DKT];
  int qi[QW], ql[QW];
#pragma unroll
  for (int w = 0; w < QW; ++w) {
    int n = MAPS == 2 ? wave * 16 + lc : (wave * QW + w) * 16 + lc;
    qi[w] = p0 + n;
    ql[w] = first_visible(a, qi[w]);
    n = n < count ? n : count - 1;
    const bf16* q = reinterpret_cast<const bf16*>(a.q) + (size_t)(row0 + n) * a.ld + (head * MAPS + (MAPS == 2 ? w : 0)) * D;
    float v[DKT][8], s = 0.f;
#pragma unroll
    for (int m = 0; m < DKT; ++m) {
      const int d = m * 32 + lg * 8;
      load8(q + (d < D ? d : 0), true, 8, v[m]);
#pragma unroll
      for (int e = 0; e < 8; ++e) {
        v[m][e] = d < D ? v[m][e] : 0.f;
        s = __builtin_fmaf(v[m][e], v[m][e], s);
      }
    }
    s += __shfl_xor(s, 16, 64);
    s += __shfl_xor(s, 32, 64);
    const float inv = a.q_norm ? 1.0f / sqrtf(s / (float)a.dim + a.eps) : 1.0f;
    const float* cs = a.rot ? angles_of(a, p0 + n) : nullptr;
#pragma unroll
    for (int m = 0; m < DKT; ++m) {
      const int d = m * 32 + lg * 8;
      if (a.q_norm) {
        float wq[8];
        load8(a.q_norm + (d < D ? d : 0), true, 8, wq);
#pragma unroll
        for (int e = 0; e < 8; ++e) v[m][e] = v[m][e] * inv * wq[e];
      }
      if (d < a.rot) rotate8(cs + d, v[m]);
#pragma unroll
      for (int e = 0; e < 8; ++e) qf[w][m][e] = (bf16)(v[m][e] * (a.scale * LOG2E));
    }
  }
  const int i_last = p0 + count - 1;
  const KeyRange keys(a, first_visible(a, p0));
  const int total = keys.count(i_last);
  const int w_first = p0 + wave * RW, w_last = w_first + RW - 1;       // (of this wave's rows)
  const int lo_first = first_visible(a, w_first), lo_last = first_visible(a, w_last);
  const bf16* kring = reinterpret_cast<const bf16*>(a.keys) + ((size_t)slot * a.G + g) * MAPS * a.ring_len * D;
  const bf16* vring = reinterpret_cast<const bf16*>(a.values) + ((size_t)slot * a.G + g) * a.ring_len * E;

  u32x4 kf[MAPS][DKT], vf[VIT];
  const int my_key = threadIdx.x >> 2, my_piece = (threadIdx.x & 3) * 8;
  auto fetch = [&](int nt) {
    const int row = keys.row(nt + my_key < total ? nt + my_key : total - 1);
#pragma unroll
    for (int t = 0; t < MAPS; ++t)
#pragma unroll
      for (int m = 0; m < DKT; ++m) {
        const int d = m * 32 + my_piece;
        kf[t][m] = *reinterpret_cast<const u32x4*>(kring + ((size_t)t * a.ring_len + row) * D + (d < D ? d : 0));
      }
#pragma unroll
    for (int m = 0; m < VIT; ++m) {
      const int d = m * 32 + my_piece;
      vf[m] = *reinterpret_cast<const u32x4*>(vring + (size_t)row * E + (d < E ? d : 0));
    }
  };
  f32x4 o[QW][DVT];
  float mx[QW], l[QW];
  const float sink = a.sink ? a.sink[head] * LOG2E : 0.f;
  const float far1 = a.far1 ? a.far1[head] : 0.f, far2 = a.far1 ? a.far2[head] : 0.f;
#pragma unroll
  for (int w = 0; w < QW; ++w) {
    mx[w] = a.sink ? sink : -1e30f;
    l[w] = a.sink && lg == 0 ? 1.0f : 0.f;
#pragma unroll
    for (int t = 0; t < DVT; ++t) o[w][t] = f32x4{0.f, 0.f, 0.f, 0.f};
  }
  fetch(0);
  for (int nt = 0; nt < total; nt += HT_KEYS) {
    __syncthreads();
#pragma unroll
    for (int t = 0; t < MAPS; ++t)
#pragma unroll
      for (int m = 0; m < DKT; ++m) *reinterpret_cast<u32x4*>(sk + (t * HT_KEYS + my_key) * KS + m * 32 + my_piece) = kf[t][m];
#pragma unroll
    for (int m = 0; m < VIT; ++m) *reinterpret_cast<u32x4*>(sv + my_key * VS + m * 32 + my_piece) = vf[m];
    if (MAPS == 1 && a.far1 && (int)threadIdx.x < HT_KEYS + 4 * RW - 1) {           // (positions follow each other: keep = 0)
      const int back = p0 + 4 * RW - 1 - keys.position(nt) - (int)threadIdx.x;
      far[threadIdx.x] = far1 * __log2f(1.0f + far2 * (float)(back > 0 ? back : 0));
    }
    __syncthreads();
    if (nt + HT_KEYS < total) fetch(nt + HT_KEYS);
    const int j_first = keys.position(nt), j_last = keys.position(nt + HT_KEYS - 1);
    if (j_first > w_last || (j_last < lo_first && j_first >= a.keep)) continue;       // nothing this wave's rows see
    const bool whole = j_last <= w_first && (j_first >= lo_last || j_last < a.keep);  // everything
    f32x4 s[QW][4];
#pragma unroll
    for (int t = 0; t < 4; ++t) {
#pragma unroll
      for (int w = 0; w < QW; ++w) s[w][t] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int c = 0; c < DKT; ++c) {
        bf16x8 kv[MAPS];
#pragma unroll
        for (int u = 0; u < MAPS; ++u) kv[u] = *reinterpret_cast<const bf16x8*>(sk + (u * HT_KEYS + t * 16 + lc) * KS + c * 32 + lg * 8);
#pragma unroll
        for (int w = 0; w < QW; ++w) s[w][t] = mma(kv[MAPS == 2 ? w : 0], qf[w][c], s[w][t]);
      }
    }
    if (MAPS == 1 && a.far1) {
#pragma unroll
      for (int w = 0; w < QW; ++w) {
        const float* f = far + lg * 4 + 4 * RW - 1 - ((wave * QW + w) * 16 + lc);
#pragma unroll
        for (int t = 0; t < 4; ++t)
#pragma unroll
          for (int e = 0; e < 4; ++e) s[w][t][e] -= f[t * 16 + e];
      }
    }
    if (!whole) {
#pragma unroll
      for (int t = 0; t < 4; ++t)
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          const int j = keys.position(nt + t * 16 + lg * 4 + e);
#pragma unroll
          for (int w = 0; w < QW; ++w)
            if (!(j <= qi[w] && (j >= ql[w] || j < a.keep))) s[w][t][e] = -INFINITY;
        }
    }
    bf16x8 p[QW][2];
#pragma unroll
    for (int w = 0; w < QW; ++w) {
      float top = mx[w];
#pragma unroll
      for (int t = 0; t < 4; ++t)
#pragma unroll
        for (int e = 0; e < 4; ++e) top = fmaxf(top, s[w][t][e]);
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
  float inv[QW];
#pragma unroll
  for (int w = 0; w < QW; ++w) {
    float tot = l[w];
    tot += __shfl_xor(tot, 16, 64);
    tot += __shfl_xor(tot, 32, 64);
    inv[w] = 1.0f / tot;
  }
  auto store = [&](int n, const f32x4 (&y)[DVT], float f) {
    if (n >= count) return;
    if (a.head_gate) f *= sigmoid_f32(a.head_gate[(size_t)(row0 + n) * a.H + head]);
    const bf16* gate = a.gate ? reinterpret_cast<const bf16*>(a.gate) + (size_t)(row0 + n) * a.ld + head * E : nullptr;
    bf16* out = reinterpret_cast<bf16*>(a.out) + ((size_t)(row0 + n) * a.H + head) * E;
#pragma unroll
    for (int t = 0; t < DVT; ++t) {
      const int d = t * 16 + lg * 4;
      if (d >= E) continue;
      bf16x4 z;
      if (gate) {
        const bf16x4 gv = *reinterpret_cast<const bf16x4*>(gate + d);
#pragma unroll
        for (int e = 0; e < 4; ++e) z[e] = (bf16)(y[t][e] * f / (1.0f + __expf(-(float)gv[e])));
      } else {
#pragma unroll
        for (int e = 0; e < 4; ++e) z[e] = (bf16)(y[t][e] * f);
      }
      *reinterpret_cast<bf16x4*>(out + d) = z;
    }
  };
  if constexpr (MAPS == 2) {
    float s = 0.f;
#pragma unroll
    for (int t = 0; t < DVT; ++t)
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        o[0][t][e] = o[0][t][e] * inv[0] - a.lambda * (o[1][t][e] * inv[1]);
        s = __builtin_fmaf(o[0][t][e], t * 16 + lg * 4 < E ? o[0][t][e] : 0.f, s);
      }
    s += __shfl_xor(s, 16, 64);
    s += __shfl_xor(s, 32, 64);
    store(wave * 16 + lc, o[0], (1.0f - a.diff) / sqrtf(s / (float)a.vdim + a.eps));
  } else {
#pragma unroll
    for (int w = 0; w < QW; ++w) store((wave * QW + w) * 16 + lc, o[w], inv[w]);
  }
}

// ------------------------------------------------------------------------------------------
static int check_head(const HA* args, const char* name) {
  PTA_REQUIRE(args, "%s: null arguments", name);
  const HA& a = *args;
  PTA_REQUIRE(a.dtype == PTA_BF16 || a.dtype == PTA_FP32, "%s: unknown type %d", name, a.dtype);
  PTA_REQUIRE(a.rows > 0 && a.G > 0 && a.H > 0 && a.H % a.G == 0 && (a.maps == 1 || a.maps == 2), "%s: rows %d, heads %d on %d, maps %d", name,
              a.rows, a.H, a.G, a.maps);
  PTA_REQUIRE(a.D > 0 && a.D <= 512 && a.D % 8 == 0 && a.E > 0 && a.E <= 512 && a.E % 8 == 0 && a.dim > 0 && a.dim <= a.D && a.vdim > 0 &&
              a.vdim <= a.E, "%s: head sizes %d and %d (multiples of 8 up to 512)", name, a.D, a.E);
  PTA_REQUIRE(a.q && a.k && a.v && pta_aligned(a.q, 16) && pta_aligned(a.k, 16) && pta_aligned(a.v, 16) && a.ld % 8 == 0,
              "%s: null or unaligned projection, rows of %d", name, a.ld);
  PTA_REQUIRE(pta_aligned(a.q_norm, 16) && pta_aligned(a.k_norm, 16), "%s: unaligned norm weight", name);
  PTA_REQUIRE(a.rot == 0 || (a.rot > 0 && a.rot % 8 == 0 && a.rot <= a.D && a.cos_sin && a.positions > 0), "%s: %d rotated features", name, a.rot);
  PTA_REQUIRE(a.window > 0 && a.keep >= 0 && a.chunk >= 0 && (a.chunk == 0 || a.keep == 0), "%s: window %d, keep %d, chunk %d", name, a.window,
              a.keep, a.chunk);
  PTA_REQUIRE(!a.far1 || (a.far2 && a.keep == 0 && a.maps == 1), "%s: a penalty of the distance needs both of its numbers, single maps and no kept positions",
              name);
  PTA_REQUIRE(a.keys && a.values && pta_aligned(a.keys, 16) && pta_aligned(a.values, 16) && a.ring_len > a.keep && a.slot && a.pos,
              "%s: the cache (%d rows) or the rows' places are missing", name, a.ring_len);
  return PTA_OK;
}

static int lanes_per_key(int n) { return n <= 32 ? 4 : n <= 64 ? 8 : n <= 128 ? 16 : n <= 256 ? 32 : 64; }

template <class F>
static void with_lanes(int n, F f) {
  switch (lanes_per_key(n)) {
    case 4: f(std::integral_constant<int, 4>{}); break;
    case 8: f(std::integral_constant<int, 8>{}); break;
    case 16: f(std::integral_constant<int, 16>{}); break;
    case 32: f(std::integral_constant<int, 32>{}); break;
    default: f(std::integral_constant<int, 64>{});
  }
}

template <typename T, int RG, int MAPS>
static void launch_rows_for(const HA& a, int fused, float* po, float* pml, hipStream_t s) {
  const int groups = (a.H / a.G + RG - 1) / RG;
  const dim3 grid((unsigned)((size_t)a.rows * a.G * groups * a.splits));
  with_lanes(a.D > a.E ? a.D : a.E, [&](auto lanes) {
    constexpr int L = decltype(lanes)::value;
    if constexpr (MAPS == 1) {
      if (a.far1 || a.conv.ring) {
        hipLaunchKernelGGL((head_rows_kernel<T, RG, MAPS, L, true>), grid, dim3(256), 0, s, a, fused, groups, po, pml);
        return;
      }
    }
    hipLaunchKernelGGL((head_rows_kernel<T, RG, MAPS, L, false>), grid, dim3(256), 0, s, a, fused, groups, po, pml);
  });
}

template <typename T>
static void launch_rows(const HA& a, int fused, float* po, float* pml, hipStream_t s) {
  const int R = a.H / a.G;
  if (a.maps == 2) {
    if (R == 1) launch_rows_for<T, 1, 2>(a, fused, po, pml, s);
    else launch_rows_for<T, 2, 2>(a, fused, po, pml, s);
  } else if (R == 1) launch_rows_for<T, 1, 1>(a, fused, po, pml, s);
  else if (R == 2) launch_rows_for<T, 2, 1>(a, fused, po, pml, s);
  else launch_rows_for<T, 4, 1>(a, fused, po, pml, s);
}

extern "C" int pta_head_append(const HA* args, pta_stream_t stream) {
  const int rc = check_head(args, "pta_head_append");
  if (rc) return rc;
  const HA& a = *args;
  with_lanes(a.D, [&](auto lanes) {
    constexpr int L = decltype(lanes)::value;
    if (a.dtype == PTA_BF16) hipLaunchKernelGGL((head_append_kernel<bf16, L>), dim3(a.rows), dim3(256), 0, (hipStream_t)stream, a);
    else hipLaunchKernelGGL((head_append_kernel<float, L>), dim3(a.rows), dim3(256), 0, (hipStream_t)stream, a);
  });
  PTA_CHECK_LAUNCH("pta_head_append");
  return PTA_OK;
}

template <int DKT, int DVT, int MAPS>
static int launch_tiles(const HA& a, hipStream_t s) {
  constexpr size_t smem = head_tile_smem<DKT, DVT, MAPS>();
  static_assert(smem <= 160 * 1024, "LDS");
  PTA_REQUIRE(smem <= 64 * 1024 || hipFuncSetAttribute((const void*)head_tile_kernel<DKT, DVT, MAPS>, hipFuncAttributeMaxDynamicSharedMemorySize,
                                                       (int)smem) == hipSuccess, "pta_head_attention: %zu bytes of LDS refused", smem);
  hipLaunchKernelGGL((head_tile_kernel<DKT, DVT, MAPS>), dim3(a.H, a.tiles, MAPS), dim3(256), smem, s, a);
  return PTA_OK;
}

template <int DKT, int MAPS>
static int launch_tiles_for(const HA& a, hipStream_t s) {
  if (a.E <= 64) return launch_tiles<DKT, 4, MAPS>(a, s);
  if (a.E <= 128) return launch_tiles<DKT, 8, MAPS>(a, s);
  return launch_tiles<DKT, 16, MAPS>(a, s);
}

template <int MAPS>
static int launch_tiles_all(const HA& a, hipStream_t s) {
  if (a.D <= 64) return launch_tiles_for<2, MAPS>(a, s);
  if (a.D <= 128) return launch_tiles_for<4, MAPS>(a, s);
  return launch_tiles_for<8, MAPS>(a, s);
}

static int check_result(const HA& a, const char* name) {
  PTA_REQUIRE(a.out && pta_aligned(a.out, 16), "%s: the output is missing or unaligned", name);
  PTA_REQUIRE(!a.gate || pta_aligned(a.gate, 16), "%s: unaligned gate", name);
  PTA_REQUIRE(a.maps == 1 || !a.sink, "%s: sinks belong to single maps", name);
  return PTA_OK;
}

extern "C" int pta_head_attention(const HA* args, pta_stream_t stream) {
  const char* name = "pta_head_attention";
  int rc = check_head(args, name);
  if (!rc) rc = check_result(*args, name);
  if (rc) return rc;
  HA a = *args;
  hipStream_t s = (hipStream_t)stream;
  a.splits = 1;
  if (a.dtype == PTA_FP32) {
    launch_rows<float>(a, 0, nullptr, nullptr, s);
  } else if (a.D > 256 || a.E > 256) {
    launch_rows<bf16>(a, 0, nullptr, nullptr, s);
  } else {
    PTA_REQUIRE(a.tile_row && a.tile_count && a.tiles > 0 && a.tiles <= 65535, "%s: %d tiles (1 .. 65535)", name, a.tiles);
    rc = a.maps == 2 ? launch_tiles_all<2>(a, s) : launch_tiles_all<1>(a, s);
    if (rc) return rc;
  }
  PTA_CHECK_LAUNCH("pta_head_attention");
  return PTA_OK;
}

extern "C" size_t pta_head_attention_workspace_bytes(int rows, int H, int maps, int E, int splits) {
  if (rows <= 0 || H <= 0 || maps <= 0 || E <= 0 || splits <= 1) return 0;
  return (size_t)rows * H * maps * splits * (E + 2) * sizeof(float);
}

extern "C" int pta_head_decode(const HA* args, pta_stream_t stream) {
  const char* name = "pta_head_decode";
  int rc = check_head(args, name);
  if (!rc) rc = check_result(*args, name);
  if (rc) return rc;
  const HA& a = *args;
  PTA_REQUIRE(a.splits >= 1 && a.splits <= 64, "%s: splits %d (1 .. 64)", name, a.splits);
  if (a.conv.ring) {
    rc = check_conv(a.conv, name);
    if (rc) return rc;
    const size_t es = a.dtype == PTA_BF16 ? 2 : 4;
    PTA_REQUIRE(a.maps == 1 && !a.conv.silu && a.conv.channels == (a.H + a.G) * a.D + a.G * a.E && (const char*)a.k == (const char*)a.q + es * a.H * a.D &&
                (const char*)a.v == (const char*)a.k + es * a.G * a.D, "%s: the convolution takes q | k | v of single maps", name);
  }
  const size_t need = pta_head_attention_workspace_bytes(a.rows, a.H, a.maps, a.E, a.splits);
  PTA_REQUIRE(a.splits == 1 || (a.workspace && a.workspace_bytes >= need), "%s: the workspace needs %zu bytes", name, need);
  hipStream_t s = (hipStream_t)stream;
  float* po = (float*)a.workspace;
  float* pml = po ? po + (size_t)a.rows * a.H * a.maps * a.splits * a.E : nullptr;
  const dim3 heads((unsigned)((size_t)a.rows * a.H));
  if (a.dtype == PTA_BF16) launch_rows<bf16>(a, 1, po, pml, s);
  else launch_rows<float>(a, 1, po, pml, s);
  if (a.splits > 1) {
    if (a.dtype == PTA_BF16 && a.maps == 2) hipLaunchKernelGGL((head_merge_kernel<bf16, 2>), heads, dim3(256), 0, s, a, po, pml);
    else if (a.dtype == PTA_BF16) hipLaunchKernelGGL((head_merge_kernel<bf16, 1>), heads, dim3(256), 0, s, a, po, pml);
    else if (a.maps == 2) hipLaunchKernelGGL((head_merge_kernel<float, 2>), heads, dim3(256), 0, s, a, po, pml);
    else hipLaunchKernelGGL((head_merge_kernel<float, 1>), heads, dim3(256), 0, s, a, po, pml);
  }
  PTA_CHECK_LAUNCH("pta_head_decode");
  return PTA_OK;
}
