// Recurrences over a matrix memory per head, S <- decay S + weight k v^T, o = S^T q, that run in chunks on the matrix unit:
// mLSTM (exponential gates under a running maximum, a normaliser beside S) and the state-space recurrence of Mamba-2
// (decay and weight from one step size, keys and queries shared by groups of heads, a direct term).
#pragma once
#include "hybrid.h"
#include <type_traits>

constexpr int SL = PTA_MLSTM_SLICE;
static_assert(PTA_SSD_SLICE == SL, "one layout of S");

// log input gate and log forget gate from their pre-activations
__device__ __forceinline__ float log_input_gate(float z, float cap) { return cap * tanhf(z / cap); }
__device__ __forceinline__ float log_forget_gate(float z, float cap) {
  const float c = cap * tanhf(z / cap);
  return fminf(c, 0.f) - log1pf(expf(-fabsf(c)));                        // log sigmoid
}
__device__ __forceinline__ float softplus_f32(float z) { return fmaxf(z, 0.f) + log1pf(expf(-fabsf(z))); }

// What the two kinds differ in.  A slice of S is followed by its copy of the normaliser and the maximum where there are such.
template <class Args> struct Memory;
template <> struct Memory<pta_mlstm_args> {
  static constexpr bool SSD = false;
  __host__ __device__ static size_t slice(int D) { return ((size_t)D * SL + D + 2 + 3) / 4 * 4; }
  __host__ __device__ static size_t part(int D) { return slice(D); }                            // what a segment leaves of a slice
  __device__ static const bf16* keys(const pta_mlstm_args& a, int head) { return reinterpret_cast<const bf16*>(a.k) + (size_t)head * a.D; }
  __device__ static const bf16* queries(const pta_mlstm_args& a, int head) { return reinterpret_cast<const bf16*>(a.q) + (size_t)head * a.D; }
  __device__ static const bf16* values(const pta_mlstm_args& a) { return reinterpret_cast<const bf16*>(a.v); }
  __device__ static float* results(const pta_mlstm_args& a) { return a.o; }
};
template <> struct Memory<pta_ssd_args> {
  static constexpr bool SSD = true;
  __host__ __device__ static size_t slice(int D) { return (size_t)D * SL; }
  __host__ __device__ static size_t part(int D) { return (size_t)D * SL + 4; }                  // S and the sum of the log decays
  __device__ static const bf16* keys(const pta_ssd_args& a, int head) { return reinterpret_cast<const bf16*>(a.b) + (size_t)(head / (a.H / a.G)) * a.D; }
  __device__ static const bf16* queries(const pta_ssd_args& a, int head) { return reinterpret_cast<const bf16*>(a.c) + (size_t)(head / (a.H / a.G)) * a.D; }
  __device__ static const bf16* values(const pta_ssd_args& a) { return reinterpret_cast<const bf16*>(a.x); }
  __device__ static float* results(const pta_ssd_args& a) { return a.y; }
};

// ------------------------------------------------------------------------------------------
// In chunks of CT tokens on the matrix unit (bf16, D <= 32 * DT), as mLSTM needs it: a workgroup per (sequence, head, CE value
// columns = two slices, segment).  With b_t the running sum of the chunk's log forget gates, a_s = i_s - b_s and
// M_t = max(m_prev, max_{s <= t} a_s), unrolling the recurrence gives m_t = b_t + M_t and
//   o_t ~ sum_{s <= t} exp(a_s - M_t) (q_t . k_s) v_s + exp(m_prev - M_t) S_prev^T q_t      (n . q likewise)
//   S  <- exp(m_prev - M_C) S_prev + sum_s exp(a_s - M_C) k_s v_s^T
// The state-space recurrence is the same with m = 0, exp(i_s) = dt_s and f = -exp(A) dt: M_t = -b_t, no normaliser, no scale.
// Everything but the projections is held in fp32; where such a value has to enter the bf16 matrix unit (the weighted
// products, the weighted values, S) it goes in as the sum of two bf16 numbers, i.e. with 16 bits.
//
// Long sequences are cut into segments that run side by side.  A first launch (OUTPUTS = false) leaves in `parts` what each
// segment but the last adds to the state (from an empty one; the first segment from the sequence's own), its m and the sum
// of its log forget gates; in the second launch a segment puts the ones before it together,
//   m' = max(m + B_i, m_i),  S' = exp(m + B_i - m') S + exp(m_i - m') S_i,
// and goes on from there.  Place 0 of `parts` keeps the state the sequence came with: the last segment overwrites it.
//
// Wave w computes outputs of tokens 16 (w % 4) .. + 15 (as columns: P^T = K Q^T, O^T = V^T P^T + S^T Q^T; with eight waves two
// share the tokens and halve the value columns) and owns rows d = w * DW .. of S in its accumulators.  The transposed values hold their tokens in the order in which a lane of the
// product P^T holds them (key 4 x + e of the first sixteen of 32 in place 8 x + e, of the second in 8 x + 4 + e); the
// transposed keys, and the weighted values beside them, in plain order.  The next chunk's rows are requested while a chunk
// is worked on.
// ------------------------------------------------------------------------------------------
constexpr int CT = 64, CE = 2 * SL;
constexpr int CS = CT + 8;

template <int DT> struct ChunkShape {
  static constexpr int DM = DT * 32, KS = DM + 8, CH = DM / 8;
  static constexpr int NW = DT >= 4 ? 8 : 4, THREADS = NW * 64;       // waves
  static constexpr int JT = 16 / NW;                                  // 16-column tiles of the outputs per wave
  static constexpr int ST = (DM / NW + 15) / 16;                      // 16-row tiles of S per wave
  static constexpr int DW = ST * 16, DS = DW * NW, SS = DS + 8;       // DS >= DM rows of S in all
  static constexpr int KT = DS * CS + DS;                             // transposed keys: row d starts at d * CS + (d / 8) * 8
  static constexpr size_t lds = 2 * ((size_t)CT * KS + KT + CE * CS + 2 * CE * (size_t)(SS > CS ? SS : CS));
};

// VEC: D and E multiples of 8 and everything 16-byte aligned - whole pieces, requested without a branch (a load in a branch
// is waited for at its end): rows past the chunk and columns past the sizes repeat others.  That is harmless in keys and
// values of rows (their weights are zero) and in key columns (they only reach rows of S that are never read); queries and
// value columns are zeroed.
template <class Args, int DT, bool OUTPUTS, bool VEC>
__global__ __launch_bounds__(ChunkShape<DT>::THREADS) void memory_chunk_kernel(Args a, int segment, int segments, float* parts) {
  typedef ChunkShape<DT> C;
  typedef Memory<Args> Kind;
  constexpr bool SSD = Kind::SSD;
  constexpr int DM = C::DM, KS = C::KS, CH = C::CH, ST = C::ST, DW = C::DW, DS = C::DS, SS = C::SS, THREADS = C::THREADS, JT = C::JT;
  constexpr int VV = 8 / C::NW, VC = VV * 8;                          // 8-column pieces and columns of the values a thread stages
  constexpr int IPT = (CT / 2 * CH + THREADS - 1) / THREADS;                      // (pair of keys, 16-byte piece) items per thread
  extern __shared__ __align__(16) unsigned char smem[];
  bf16* sk = reinterpret_cast<bf16*>(smem);                           // [CT][KS] keys
  bf16* skt = sk + CT * KS;                                           // keys transposed
  bf16* svt = skt + C::KT;                                            // [CE][CS] values transposed, permuted
  bf16* big = svt + CE * CS;
  bf16* ss_hi = big;                                                  // [CE][SS] S transposed, two parts
  bf16* ss_lo = big + CE * SS;
  bf16* sw_hi = big;                                                  // [CE][CS] weighted values, over S once that is read
  bf16* sw_lo = big + CE * CS;
  __shared__ __align__(16) float s_n[DM], s_a[CT], s_M[CT], s_b[CT], s_w[CT];
  __shared__ float s_m;
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  int lane = threadIdx.x & 63, lg = lane >> 4, lc = lane & 15;
  const int slices = (a.E + SL - 1) / SL, groups = (slices + 1) / 2;
  int blk = blockIdx.x;
  const int grp = blk % groups; blk /= groups;
  const int head = blk % a.H; blk /= a.H;
  const int seg = blk % segments, seq = blk / segments;
  const int total = a.seq_count[seq], first = seg * segment;
  const bool final_seg = first + segment >= total;                    // ... of its sequence
  if (first >= total || (!OUTPUTS && final_seg)) return;
  const int D = a.D, E = a.E, count = total - first < segment ? total - first : segment;
  const int row_s = a.seq_row[seq], row0 = row_s + first;
  const int e0 = grp * CE, ecols = E - e0 < CE ? E - e0 : CE;
  const size_t st_per = Kind::slice(D), per = Kind::part(D), first_slice = (size_t)head * slices + grp * 2;
  const size_t whole = (size_t)a.H * slices * per;
  float* st = a.state + ((size_t)a.slot[row_s] * a.H * slices + first_slice) * st_per;
  float* part = parts + (size_t)seq * segments * whole + first_slice * per;     // place j: what segment j starts from (j = 0), or segment j - 1 left
  const bool second = grp * 2 + 1 < slices, several = total > segment;
  const float qscale = SSD ? 1.0f : 1.0f / sqrtf((float)D);
  float dt_bias = 0.f, decay_rate = 0.f, direct = 0.f;                // state space: of this head
  if constexpr (SSD) {
    dt_bias = a.dt_bias[head];
    decay_rate = -expf(a.a_log[head]);
    direct = a.skip[head];
  }

  // ---- the chunk's rows on their way to LDS (keys, values), to registers (queries) and the gates
  u32x4 kr[IPT][2], vr[VV], qr[DT];
  float zi, zf;
  // (a uniform base per chunk and a 32-bit offset per lane)
  auto row8 = [&](const bf16* base, int r, int at, int left) {
    const bf16* src = base + (unsigned)(r * a.ld + at);
    if constexpr (VEC) return *reinterpret_cast<const u32x4*>(src);
    bf16x8 z;
#pragma unroll
    for (int e = 0; e < 8; ++e) z[e] = e < left ? src[e] : (bf16)0.0f;
    return bitcast<u32x4>(z);
  };
  const u32x4 none = {0, 0, 0, 0};
  auto fetch = [&](int t0) {
    const int cnt = count - t0 < CT ? count - t0 : CT;
    const size_t rb = (size_t)row0 + t0;
    const bf16 *kb = Kind::keys(a, head) + rb * a.ld, *qb = Kind::queries(a, head) + rb * a.ld, *vb = Kind::values(a) + rb * a.ld + head * E + e0;
    if constexpr (SSD) {
      zi = a.dt[rb * a.H + head + (unsigned)((lane < cnt ? lane : cnt - 1) * a.H)];
    } else {
      const float* z = a.gates + rb * 2 * a.H + head + (unsigned)((lane < cnt ? lane : cnt - 1) * 2 * a.H);
      zi = z[0];
      zf = z[a.H];
    }
#pragma unroll
    for (int it = 0; it < IPT; ++it) {
      const int idx = threadIdx.x + it * THREADS, c = idx % CH, kp = idx / CH, left = D - c * 8;
#pragma unroll
      for (int t = 0; t < 2; ++t) {
        const int s = kp * 2 + t;
        kr[it][t] = row8(kb, s < cnt ? s : cnt - 1, left > 0 ? c * 8 : 0, left);
      }
    }
    {
      const int s = threadIdx.x & 63, c0 = wave * VC;
#pragma unroll
      for (int h = 0; h < VV; ++h) {
        const int left = ecols - c0 - h * 8;
        vr[h] = row8(vb, s < cnt ? s : cnt - 1, left > 0 ? c0 + h * 8 : 0, left);
      }
    }
    if (OUTPUTS) {
      const int t = (wave & 3) * 16 + lc;
#pragma unroll
      for (int c = 0; c < DT; ++c) {
        const int left = D - c * 32 - lg * 8;
        qr[c] = row8(qb, t < cnt ? t : cnt - 1, left > 0 ? c * 32 + lg * 8 : 0, left);
      }
    }
  };
  fetch(0);

  // ---- the state at the start.  Lane holds rows d = wave * DW + 16 i + 4 lg + 0..3 of column e = 16 j + lc
  f32x4 S[ST][4];
  float m_prev;
  const int lane_d = wave * DW + lg * 4, lane_at = lane_d * SL + lc;
  // (iper: from one slice to the next of what is addressed)
  auto each = [&](int iper, auto fn) {
    int base = lane_at;
    asm volatile("" : "+v"(base));       // the 64 offsets are made anew at every use instead of being kept in registers
#pragma unroll
    for (int i = 0; i < ST; ++i)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const bool row = lane_d + i * 16 + r < D;
        const int at = base + (i * 16 + r) * SL;
#pragma unroll
        for (int j = 0; j < 4; ++j)
          S[i][j][r] = fn(S[i][j][r], at + (j & 1) * 16 + (j >> 1) * iper, row && (j < 2 || second));
      }
  };
  {
    const bool empty = !OUTPUTS && seg > 0;
    // a segment of several starts from what the first launch kept: the state itself is overwritten by the last segment
    const bool from_part = OUTPUTS && several;
    const float* from = from_part ? part + (seg > 0 ? whole : 0) : st;
    each((int)(from_part ? per : st_per), [&](float, int at, bool there) {                     // (loads without a branch, as above)
      const float x = from[there ? at : 0];
      return there && !empty ? x : 0.f;
    });
    m_prev = 0.f;
    if constexpr (!SSD) {
      for (int d = threadIdx.x; d < DM; d += THREADS) s_n[d] = d < D && !empty ? from[(size_t)D * SL + d] : 0.f;
      m_prev = empty ? -INFINITY : from[(size_t)D * SL + D];
    }
    if (!OUTPUTS && seg == 0) {                               // keep what the sequence came with
      each((int)per, [&](float x, int at, bool there) { if (there) part[at] = x; return x; });
      if constexpr (!SSD) {
        for (int d = threadIdx.x; d < D; d += THREADS) part[(size_t)D * SL + d] = s_n[d];
        if (threadIdx.x == 0) part[(size_t)D * SL + D] = m_prev;
      }
    }
    if (OUTPUTS)
      for (int j = 2; j <= seg; ++j) {
        const float* add = part + (size_t)j * whole;
        float keep, take = 1.0f, mn = 0.f;
        if constexpr (SSD) {
          keep = expf(add[(size_t)D * SL]);
        } else {
          const float mi = add[(size_t)D * SL + D], carried = m_prev + add[(size_t)D * SL + D + 1];
          mn = fmaxf(carried, mi);
          keep = expf(carried - mn);
          take = expf(mi - mn);
        }
        each((int)per, [&](float x, int at, bool there) {
          const float y = add[there ? at : 0];
          return __builtin_fmaf(keep, x, (there ? take : 0.f) * y);
        });
        if constexpr (!SSD) {
          for (int d = threadIdx.x; d < D; d += THREADS) s_n[d] = __builtin_fmaf(keep, s_n[d], take * add[(size_t)D * SL + d]);
          m_prev = mn;
        }
      }
  }
  if (DS > DM)
    for (int idx = threadIdx.x; idx < (DS - DM) * (CS + 1); idx += THREADS) skt[DM * (CS + 1) + idx] = (bf16)0.0f;

  float b_total = 0.f;
  for (int t0 = 0; t0 < count; t0 += CT) {
    const int cnt = count - t0 < CT ? count - t0 : CT;
    const size_t rb = (size_t)row0 + t0;
    // (the many LDS addresses below are made anew in every chunk: kept in registers across chunks they spill)
    asm volatile("" : "+v"(lane));
    lg = lane >> 4;
    lc = lane & 15;
    const int tid = wave * 64 + lane;
    // ---- S in two bf16 parts, keys and values into LDS, gates
    if (OUTPUTS) {
#pragma unroll
      for (int i = 0; i < ST; ++i)
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          bf16x4 hi, lo;
#pragma unroll
          for (int r = 0; r < 4; ++r) {
            hi[r] = (bf16)S[i][j][r];
            lo[r] = (bf16)(S[i][j][r] - (float)hi[r]);
          }
          const int at = (j * 16 + lc) * SS + wave * DW + i * 16 + lg * 4;
          *reinterpret_cast<bf16x4*>(ss_hi + at) = hi;
          *reinterpret_cast<bf16x4*>(ss_lo + at) = lo;
        }
    }
#pragma unroll
    for (int it = 0; it < IPT; ++it) {
      const int idx = tid + it * THREADS, c = idx % CH, kp = idx / CH;
      if (idx >= CT / 2 * CH) break;
      if (OUTPUTS) {
        *reinterpret_cast<u32x4*>(sk + (kp * 2) * KS + c * 8) = kr[it][0];
        *reinterpret_cast<u32x4*>(sk + (kp * 2 + 1) * KS + c * 8) = kr[it][1];
      }
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        bf16* base = skt + (c * 8 + 2 * e) * CS + c * 8 + kp * 2;
        *reinterpret_cast<uint32_t*>(base) = (kr[it][0][e] & 0xffffu) | (kr[it][1][e] << 16);
        *reinterpret_cast<uint32_t*>(base + CS) = (kr[it][0][e] >> 16) | (kr[it][1][e] & 0xffff0000u);
      }
    }
    // values: thread (token s = tid % 64, columns VC * (tid / 64) ..): kept in registers for the weighted copy
    bf16x8 v8[VV];
#pragma unroll
    for (int h = 0; h < VV; ++h) v8[h] = bitcast<bf16x8>(ecols - wave * VC - h * 8 > 0 ? vr[h] : none);
    if (OUTPUTS) {
      const int s = lane, k32 = s & 31, place = (s & 32) + ((k32 & 15) >> 2) * 8 + (k32 >> 4) * 4 + (k32 & 3);
#pragma unroll
      for (int e = 0; e < VC; ++e) svt[(wave * VC + e) * CS + place] = v8[e >> 3][e & 7];
    }
    // gates of the chunk: running sums and maxima over the 64 lanes of the first wave
    if constexpr (SSD) {
      if (wave == 0) {
        const float dt = lane < cnt ? softplus_f32(zi + dt_bias) : 0.f;
        float bsum = decay_rate * dt;
#pragma unroll
        for (int o = 1; o < 64; o <<= 1) {
          const float t = __shfl_up(bsum, o, 64);
          if (lane >= o) bsum += t;
        }
        const float last = __shfl(bsum, 63, 64);
        s_a[lane] = dt;
        s_b[lane] = bsum;
        s_w[lane] = dt * expf(last - bsum);
      }
    } else if (wave == 0) {
      const float gi = lane < cnt ? log_input_gate(zi, a.cap) : -INFINITY, gf = lane < cnt ? log_forget_gate(zf, a.cap) : 0.f;
      float bsum = gf;
#pragma unroll
      for (int o = 1; o < 64; o <<= 1) {
        const float t = __shfl_up(bsum, o, 64);
        if (lane >= o) bsum += t;
      }
      const float av = gi - bsum;
      float top = av;
#pragma unroll
      for (int o = 1; o < 64; o <<= 1) {
        const float t = __shfl_up(top, o, 64);
        if (lane >= o) top = fmaxf(top, t);
      }
      top = fmaxf(top, m_prev);
      const float last = __shfl(top, 63, 64);                 // M of the whole chunk (tokens past cnt add nothing)
      s_a[lane] = av;
      s_b[lane] = bsum;
      s_M[lane] = top;
      s_w[lane] = expf(av - last);
      if (lane == 63) s_m = bsum + last;
    }
    bf16x8 qf[DT];
    if (OUTPUTS) {
#pragma unroll
      for (int c = 0; c < DT; ++c) qf[c] = bitcast<bf16x8>(D - c * 32 - lg * 8 > 0 ? qr[c] : none);
    }
    __syncthreads();
    if (t0 + CT < count) fetch(t0 + CT);

    const float m_chunk = SSD ? 0.f : s_m, M_last = SSD ? -s_b[CT - 1] : s_M[CT - 1];
    b_total += s_b[CT - 1];
    // ---- outputs of this wave's sixteen tokens
    if (OUTPUTS) {
      const int t = (wave & 3) * 16 + lc;
      const int j0 = (wave >> 2) * JT;                        // first column tile of this wave's outputs
      float nq = 0.f;
      if constexpr (!SSD) {
#pragma unroll
        for (int c = 0; c < DT; ++c)
#pragma unroll
          for (int e = 0; e < 8; ++e) nq = __builtin_fmaf((float)qf[c][e], s_n[c * 32 + lg * 8 + e], nq);
        nq += __shfl_xor(nq, 16, 64);
        nq += __shfl_xor(nq, 32, 64);
      }
      const float bt = s_b[t], Mt = SSD ? -bt : s_M[t], inter = expf(m_prev - Mt);
      f32x4 o[JT];
#pragma unroll
      for (int j = 0; j < JT; ++j) o[j] = f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int c = 0; c < DT; ++c) {
#pragma unroll
        for (int j = 0; j < JT; ++j) {
          const int at = ((j0 + j) * 16 + lc) * SS + c * 32 + lg * 8;
          o[j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(*reinterpret_cast<const bf16x8*>(ss_hi + at), qf[c], o[j], 0, 0, 0);
          o[j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(*reinterpret_cast<const bf16x8*>(ss_lo + at), qf[c], o[j], 0, 0, 0);
        }
      }
#pragma unroll
      for (int j = 0; j < JT; ++j)
#pragma unroll
        for (int r = 0; r < 4; ++r) o[j][r] *= inter;
      nq *= inter;
      float psum = 0.f;
#pragma unroll
      for (int kg = 0; kg < 2; ++kg) {
        if (kg * 32 > (wave & 3) * 16 + 15) continue;              // all of these keys come after this wave's tokens
        bf16x8 hi, lo;
#pragma unroll
        for (int h = 0; h < 2; ++h) {
          f32x4 p = {0.f, 0.f, 0.f, 0.f};
          const f32x4 as = *reinterpret_cast<const f32x4*>(s_a + kg * 32 + h * 16 + lg * 4);
          f32x4 bs = {0.f, 0.f, 0.f, 0.f};
          if constexpr (SSD) bs = *reinterpret_cast<const f32x4*>(s_b + kg * 32 + h * 16 + lg * 4);
#pragma unroll
          for (int c = 0; c < DT; ++c)
            p = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
                *reinterpret_cast<const bf16x8*>(sk + (kg * 32 + h * 16 + lc) * KS + c * 32 + lg * 8), qf[c], p, 0, 0, 0);
#pragma unroll
          for (int r = 0; r < 4; ++r) {
            const int s = kg * 32 + h * 16 + lg * 4 + r;
            const float x = SSD ? p[r] * (as[r] * __expf(s <= t ? bt - bs[r] : -INFINITY)) : p[r] * __expf(s <= t ? as[r] - Mt : -INFINITY);
            psum += x;
            hi[h * 4 + r] = (bf16)x;
            lo[h * 4 + r] = (bf16)(x - (float)hi[h * 4 + r]);
          }
        }
#pragma unroll
        for (int j = 0; j < JT; ++j) {
          const bf16x8 vf = *reinterpret_cast<const bf16x8*>(svt + ((j0 + j) * 16 + lc) * CS + kg * 32 + lg * 8);
          o[j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf, hi, o[j], 0, 0, 0);
          o[j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf, lo, o[j], 0, 0, 0);
        }
      }
      float f = 1.0f;
      if constexpr (SSD) {                                     // the direct term
        const int k32 = t & 31, place = (t & 32) + ((k32 & 15) >> 2) * 8 + (k32 >> 4) * 4 + (k32 & 3);
#pragma unroll
        for (int j = 0; j < JT; ++j)
#pragma unroll
          for (int r = 0; r < 4; ++r)
            o[j][r] = __builtin_fmaf(direct, (float)svt[((j0 + j) * 16 + lg * 4 + r) * CS + place], o[j][r]);
      } else {
        psum += __shfl_xor(psum, 16, 64);
        psum += __shfl_xor(psum, 32, 64);
        const float den = fmaxf(fabsf((nq + psum) * qscale), expf(-(bt + Mt))) + 1e-6f;
        f = qscale / den;
      }
      if (t < cnt) {
        float* dst = Kind::results(a) + (rb + t) * a.H * E + (size_t)head * E + e0;
#pragma unroll
        for (int j = 0; j < JT; ++j) {
          const int e = (j0 + j) * 16 + lg * 4;
          if (e + 4 <= ecols && (E & 3) == 0) {
            *reinterpret_cast<f32x4*>(dst + e) = f32x4{o[j][0] * f, o[j][1] * f, o[j][2] * f, o[j][3] * f};
          } else {
#pragma unroll
            for (int r = 0; r < 4; ++r)
              if (e + r < ecols) dst[e + r] = o[j][r] * f;
          }
        }
      }
      __syncthreads();                                        // S, the keys as they are and n have been read
    }

    // ---- the state at the end of the chunk
    {
      const int s = lane;
      const float w = s < cnt ? s_w[s] : 0.f;
#pragma unroll
      for (int e = 0; e < VC; ++e) {
        const float x = (float)v8[e >> 3][e & 7] * w;
        const bf16 hi = (bf16)x;
        sw_hi[(wave * VC + e) * CS + s] = hi;
        sw_lo[(wave * VC + e) * CS + s] = (bf16)(x - (float)hi);
      }
    }
    const float decay = expf(m_prev - M_last);
    if constexpr (!SSD) for (int d = tid; d < DM; d += THREADS) {
      float n = s_n[d] * decay;
#pragma unroll
      for (int s = 0; s < CT; s += 8) {
        const bf16x8 kv = *reinterpret_cast<const bf16x8*>(skt + d * CS + (d >> 3) * 8 + s);
#pragma unroll
        for (int e = 0; e < 8; ++e) n = __builtin_fmaf(s_w[s + e], (float)kv[e], n);
      }
      s_n[d] = n;
    }
    __syncthreads();
#pragma unroll
    for (int i = 0; i < ST; ++i)
#pragma unroll
      for (int j = 0; j < 4; ++j)
#pragma unroll
        for (int r = 0; r < 4; ++r) S[i][j][r] *= decay;
#pragma unroll
    for (int kg = 0; kg < 2; ++kg) {
      bf16x8 wh[4], wl[4];
#pragma unroll
      for (int j = 0; j < 4; ++j) {
        const int at = (j * 16 + lc) * CS + kg * 32 + lg * 8;
        wh[j] = *reinterpret_cast<const bf16x8*>(sw_hi + at);
        wl[j] = *reinterpret_cast<const bf16x8*>(sw_lo + at);
      }
#pragma unroll
      for (int i = 0; i < ST; ++i) {
        const int d = wave * DW + i * 16 + lc;
        const bf16x8 kf = *reinterpret_cast<const bf16x8*>(skt + d * CS + (d >> 3) * 8 + kg * 32 + lg * 8);
#pragma unroll
        for (int j = 0; j < 4; ++j) {
          S[i][j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf, wh[j], S[i][j], 0, 0, 0);
          S[i][j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf, wl[j], S[i][j], 0, 0, 0);
        }
      }
    }
    m_prev = m_chunk;
    __syncthreads();                                          // before the next chunk's data replaces this one's
  }
  if (!OUTPUTS || final_seg) {
    float* to = OUTPUTS ? st : part + (size_t)(seg + 1) * whole;
    each((int)(OUTPUTS ? st_per : per), [&](float x, int at, bool there) { if (there) to[at] = x; return x; });
    if constexpr (SSD) {
      if (!OUTPUTS && (int)threadIdx.x < (second ? 2 : 1)) to[threadIdx.x * per + (size_t)D * SL] = b_total;
    } else for (int h = 0; h < (second ? 2 : 1); ++h) {
      for (int d = threadIdx.x; d < D; d += THREADS) to[h * per + (size_t)D * SL + d] = s_n[d];
      if (threadIdx.x == 0) {
        to[h * per + (size_t)D * SL + D] = m_prev;
        if (!OUTPUTS) to[h * per + (size_t)D * SL + D + 1] = b_total;
      }
    }
  }
}

// Segments of a pass: as many as fill the machine with workgroups, of at least two chunks each.
template <class Args>
static int chunk_segments(const Args& a, int* length) {
  const int base = a.seqs * a.H * (((a.E + SL - 1) / SL + 1) / 2);
  int n = (256 + base - 1) / base;
  n = n > 16 ? 16 : n;
  int len = (a.longest + n - 1) / n;
  len = (len + CT - 1) / CT * CT;
  if (len < 2 * CT) len = 2 * CT;
  *length = len;
  return (a.longest + len - 1) / len;
}

template <class Args>
static size_t chunk_workspace_bytes(const Args* args) {
  if (!args || args->dtype != PTA_BF16 || !args->chunked || args->D > 256 || args->seqs <= 0 || args->longest <= 0 || args->H <= 0 || args->E <= 0) return 0;
  int len;
  const int n = chunk_segments(*args, &len);
  return n > 1 ? (size_t)args->seqs * n * args->H * ((args->E + SL - 1) / SL) * Memory<Args>::part(args->D) * sizeof(float) : 0;
}

template <class Args, int DT, bool VEC>
static int launch_chunk(const Args& a, hipStream_t s, const char* name) {
  static bool ready = false;
  constexpr size_t smem = ChunkShape<DT>::lds;
  static_assert(smem + 4096 <= 160 * 1024, "LDS");
  const void *outs = (const void*)memory_chunk_kernel<Args, DT, true, VEC>, *sums = (const void*)memory_chunk_kernel<Args, DT, false, VEC>;
  if (!ready) {
    PTA_REQUIRE(hipFuncSetAttribute(outs, hipFuncAttributeMaxDynamicSharedMemorySize, (int)smem) == hipSuccess &&
                hipFuncSetAttribute(sums, hipFuncAttributeMaxDynamicSharedMemorySize, (int)smem) == hipSuccess,
                "%s: cannot reserve %zu bytes of LDS", name, smem);
    ready = true;
  }
  int length;
  const int segments = chunk_segments(a, &length);
  const size_t need = chunk_workspace_bytes(&a);
  PTA_REQUIRE(segments == 1 || (a.workspace && a.workspace_bytes >= need), "%s: the workspace needs %zu bytes", name, need);
  const int slices = (a.E + SL - 1) / SL;
  const dim3 grid(a.seqs * a.H * ((slices + 1) / 2) * segments);
  if (segments > 1)
    hipLaunchKernelGGL((memory_chunk_kernel<Args, DT, false, VEC>), grid, dim3(ChunkShape<DT>::THREADS), smem, s, a, length, segments, (float*)a.workspace);
  hipLaunchKernelGGL((memory_chunk_kernel<Args, DT, true, VEC>), grid, dim3(ChunkShape<DT>::THREADS), smem, s, a, length, segments, (float*)a.workspace);
  return PTA_OK;
}
