// Matrix memory (mLSTM): the recurrence token by token, the same in chunks on the matrix unit, and the per-head norm
// with the output gate.
#include "hybrid.h"

typedef pta_mlstm_args MA;
constexpr int SL = PTA_MLSTM_SLICE;

extern "C" size_t pta_mlstm_state_floats(int H, int D, int E) {
  if (H <= 0 || D <= 0 || E <= 0) return 0;
  const size_t slice = ((size_t)D * SL + D + 2 + 3) / 4 * 4;             // slices start on 16-byte boundaries
  return (size_t)H * ((E + SL - 1) / SL) * slice;
}
__device__ __forceinline__ size_t slice_floats(int D) { return ((size_t)D * SL + D + 2 + 3) / 4 * 4; }

// log input gate and log forget gate from their pre-activations
__device__ __forceinline__ float log_input_gate(float z, float cap) { return cap * tanhf(z / cap); }
__device__ __forceinline__ float log_forget_gate(float z, float cap) {
  const float c = cap * tanhf(z / cap);
  return fminf(c, 0.f) - log1pf(expf(-fabsf(c)));                        // log sigmoid
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
  const size_t per = slice_floats(D);
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

// ------------------------------------------------------------------------------------------
// In chunks of CT tokens on the matrix unit (bf16, D <= 32 * DT): a workgroup per (sequence, head, CE value
// columns = two slices, segment).  With b_t the running sum of the chunk's log forget gates, a_s = i_s - b_s and
// M_t = max(m_prev, max_{s <= t} a_s), unrolling the recurrence gives m_t = b_t + M_t and
//   o_t ~ sum_{s <= t} exp(a_s - M_t) (q_t . k_s) v_s + exp(m_prev - M_t) S_prev^T q_t      (n . q likewise)
//   S  <- exp(m_prev - M_C) S_prev + sum_s exp(a_s - M_C) k_s v_s^T
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
template <int DT, bool OUTPUTS, bool VEC>
__global__ __launch_bounds__(ChunkShape<DT>::THREADS) void mlstm_chunk_kernel(MA a, int segment, int segments, float* parts) {
  typedef ChunkShape<DT> C;
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
  const size_t per = slice_floats(D);
  const size_t pair_at = ((size_t)head * slices + grp * 2) * per, whole = (size_t)a.H * slices * per;
  float* st = a.state + (size_t)a.slot[row_s] * whole + pair_at;
  float* part = parts + (size_t)seq * segments * whole + pair_at;     // place j: what segment j starts from (j = 0), or segment j - 1 left
  const bool second = grp * 2 + 1 < slices, several = total > segment;
  const float qscale = 1.0f / sqrtf((float)D);

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
    const bf16 *kb = reinterpret_cast<const bf16*>(a.k) + rb * a.ld + head * D, *qb = reinterpret_cast<const bf16*>(a.q) + rb * a.ld + head * D,
               *vb = reinterpret_cast<const bf16*>(a.v) + rb * a.ld + head * E + e0;
    {
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
  const int lane_d = wave * DW + lg * 4, lane_at = lane_d * SL + lc, iper = (int)per;
  auto each = [&](auto fn) {
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
    const float* from = OUTPUTS && several ? part + (seg > 0 ? whole : 0) : st;
    each([&](float, int at, bool there) {                     // (loads without a branch, as above)
      const float x = from[there ? at : 0];
      return there && !empty ? x : 0.f;
    });
    for (int d = threadIdx.x; d < DM; d += THREADS) s_n[d] = d < D && !empty ? from[(size_t)D * SL + d] : 0.f;
    m_prev = empty ? -INFINITY : from[(size_t)D * SL + D];
    if (!OUTPUTS && seg == 0) {                               // keep what the sequence came with
      each([&](float x, int at, bool there) { if (there) part[at] = x; return x; });
      for (int d = threadIdx.x; d < D; d += THREADS) part[(size_t)D * SL + d] = s_n[d];
      if (threadIdx.x == 0) part[(size_t)D * SL + D] = m_prev;
    }
    if (OUTPUTS)
      for (int j = 2; j <= seg; ++j) {
        const float* add = part + (size_t)j * whole;
        const float mi = add[(size_t)D * SL + D], carried = m_prev + add[(size_t)D * SL + D + 1];
        const float mn = fmaxf(carried, mi), keep = expf(carried - mn), take = expf(mi - mn);
        each([&](float x, int at, bool there) {
          const float y = add[there ? at : 0];
          return __builtin_fmaf(keep, x, (there ? take : 0.f) * y);
        });
        for (int d = threadIdx.x; d < D; d += THREADS) s_n[d] = __builtin_fmaf(keep, s_n[d], take * add[(size_t)D * SL + d]);
        m_prev = mn;
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
    if (wave == 0) {
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

    const float m_chunk = s_m, M_last = s_M[CT - 1];
    b_total += s_b[CT - 1];
    // ---- outputs of this wave's sixteen tokens
    if (OUTPUTS) {
      const int t = (wave & 3) * 16 + lc;
      const int j0 = (wave >> 2) * JT;                        // first column tile of this wave's outputs
      float nq = 0.f;
#pragma unroll
      for (int c = 0; c < DT; ++c)
#pragma unroll
        for (int e = 0; e < 8; ++e) nq = __builtin_fmaf((float)qf[c][e], s_n[c * 32 + lg * 8 + e], nq);
      nq += __shfl_xor(nq, 16, 64);
      nq += __shfl_xor(nq, 32, 64);
      const float Mt = s_M[t], bt = s_b[t], inter = expf(m_prev - Mt);
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
#pragma unroll
          for (int c = 0; c < DT; ++c)
            p = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
                *reinterpret_cast<const bf16x8*>(sk + (kg * 32 + h * 16 + lc) * KS + c * 32 + lg * 8), qf[c], p, 0, 0, 0);
#pragma unroll
          for (int r = 0; r < 4; ++r) {
            const int s = kg * 32 + h * 16 + lg * 4 + r;
            const float x = p[r] * __expf(s <= t ? as[r] - Mt : -INFINITY);
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
      psum += __shfl_xor(psum, 16, 64);
      psum += __shfl_xor(psum, 32, 64);
      const float den = fmaxf(fabsf((nq + psum) * qscale), expf(-(bt + Mt))) + 1e-6f;
      const float f = qscale / den;
      if (t < cnt) {
        float* dst = a.o + (rb + t) * a.H * E + (size_t)head * E + e0;
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
    for (int d = tid; d < DM; d += THREADS) {
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
    each([&](float x, int at, bool there) { if (there) to[at] = x; return x; });
    for (int h = 0; h < (second ? 2 : 1); ++h) {
      for (int d = threadIdx.x; d < D; d += THREADS) to[h * per + (size_t)D * SL + d] = s_n[d];
      if (threadIdx.x == 0) {
        to[h * per + (size_t)D * SL + D] = m_prev;
        if (!OUTPUTS) to[h * per + (size_t)D * SL + D + 1] = b_total;
      }
    }
  }
}

// Segments of a pass: as many as fill the machine with workgroups, of at least two chunks each.
static int chunk_segments(const MA& a, int* length) {
  const int base = a.seqs * a.H * (((a.E + SL - 1) / SL + 1) / 2);
  int n = (256 + base - 1) / base;
  n = n > 16 ? 16 : n;
  int len = (a.longest + n - 1) / n;
  len = (len + CT - 1) / CT * CT;
  if (len < 2 * CT) len = 2 * CT;
  *length = len;
  return (a.longest + len - 1) / len;
}

extern "C" size_t pta_mlstm_workspace_bytes(const MA* args) {
  if (!args || args->dtype != PTA_BF16 || !args->chunked || args->D > 256 || args->seqs <= 0 || args->longest <= 0 || args->H <= 0 || args->E <= 0) return 0;
  int len;
  const int n = chunk_segments(*args, &len);
  return n > 1 ? (size_t)args->seqs * n * pta_mlstm_state_floats(args->H, args->D, args->E) * sizeof(float) : 0;
}

template <int DT, bool VEC>
static int launch_chunk(const MA& a, hipStream_t s) {
  static bool ready = false;
  constexpr size_t smem = ChunkShape<DT>::lds;
  static_assert(smem + 4096 <= 160 * 1024, "LDS");
  const void *outs = (const void*)mlstm_chunk_kernel<DT, true, VEC>, *sums = (const void*)mlstm_chunk_kernel<DT, false, VEC>;
  if (!ready) {
    PTA_REQUIRE(hipFuncSetAttribute(outs, hipFuncAttributeMaxDynamicSharedMemorySize, (int)smem) == hipSuccess &&
                hipFuncSetAttribute(sums, hipFuncAttributeMaxDynamicSharedMemorySize, (int)smem) == hipSuccess,
                "pta_mlstm: cannot reserve %zu bytes of LDS", smem);
    ready = true;
  }
  int length;
  const int segments = chunk_segments(a, &length);
  const size_t need = pta_mlstm_workspace_bytes(&a);
  PTA_REQUIRE(segments == 1 || (a.workspace && a.workspace_bytes >= need), "pta_mlstm: the workspace needs %zu bytes", need);
  const int slices = (a.E + SL - 1) / SL;
  const dim3 grid(a.seqs * a.H * ((slices + 1) / 2) * segments);
  if (segments > 1)
    hipLaunchKernelGGL((mlstm_chunk_kernel<DT, false, VEC>), grid, dim3(ChunkShape<DT>::THREADS), smem, s, a, length, segments, (float*)a.workspace);
  hipLaunchKernelGGL((mlstm_chunk_kernel<DT, true, VEC>), grid, dim3(ChunkShape<DT>::THREADS), smem, s, a, length, segments, (float*)a.workspace);
  return PTA_OK;
}

template <int DT>
static int launch_chunk(const MA& a, bool vec, hipStream_t s) {
  return vec ? launch_chunk<DT, true>(a, s) : launch_chunk<DT, false>(a, s);
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
    if (a.D <= 32) rc = launch_chunk<1>(a, vec, s);
    else if (a.D <= 64) rc = launch_chunk<2>(a, vec, s);
    else if (a.D <= 128) rc = launch_chunk<4>(a, vec, s);
    else rc = launch_chunk<8>(a, vec, s);
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
