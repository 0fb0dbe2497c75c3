/*
 * poptransformer_hybrid.h - C ABI of libpoptransformer_hybrid.so (gfx950 / MI355X).
 *
 * Kernels of decoders whose layers mix attention over a window with recurrent (matrix memory) layers and whose
 * residual stream is kept in 32-bit, possibly as several parallel streams.  Activations and weights are bf16
 * (PTA_BF16: matrix unit, fp32 accumulation) or fp32 (PTA_FP32: true 32-bit throughout).
 *
 * A call works on the ROWS of a pass: row r is one token of the sequence that holds cache slot slot[r], at position
 * pos[r] of that sequence.  A pass may mix rows of many sequences; the rows of one sequence follow each other in order
 * of position.  Nothing else ties the rows together: a decode step is a pass with one row per sequence, a prompt is a
 * pass (or several) with many.
 *
 * Rules: as in poptransformer_hip.h (device pointers, nothing allocated or synchronised, PTA_* status codes,
 * pta_hybrid_last_error() for the message).
 */
#ifndef POPTRANSFORMER_HYBRID_H
#define POPTRANSFORMER_HYBRID_H

#include <stddef.h>
#include <stdint.h>
#include "poptransformer_hip.h"

#ifdef __cplusplus
extern "C" {
#endif

enum { PTA_BF16 = 0, PTA_FP32 = 1 };

const char* pta_hybrid_last_error(void);

/* ---- Linear layers -----------------------------------------------------------------------------------------------
 * Y = X @ W^T with fp32 accumulation and an fp32 epilogue that rounds once, where a value is stored.
 * bf16 weights are tiled once with pta_bf16_tile; fp32 weights stay row-major [N, K] (K a multiple of 4, 16-byte
 * aligned).  N may exceed n_main + tail_count: the channels past them are padding and go nowhere. */
size_t pta_bf16_tiled_bytes(int N, int K);
int pta_bf16_tile(const uint16_t* w, void* tiled, int N, int K, pta_stream_t stream);

enum { PTA_PAIR_NONE = 0, PTA_PAIR_SWIGLU = 1, PTA_PAIR_CLAMPED = 2 };

typedef struct pta_wide_linear_args {
  int dtype;              /* PTA_BF16 / PTA_FP32: type of X and W                                                  */
  const void* X;          /* [M, K]                                                                                */
  int M, K, N;            /* K a multiple of 8; 1 <= M <= 4096                                                     */
  const void* W;          /* the weight; of a pair the gate                                                        */
  const void* W2;         /* of a pair the up weight, same shape                                                   */
  int pair;               /* PTA_PAIR_*: SWIGLU u * g * sigmoid(g);
                             CLAMPED with g' = min(g, limit), u' = clamp(u, -limit, limit): g' sigmoid(slope g') (u' + 1) */
  float limit, slope;
  float cap;              /* > 0: y = cap * tanh(y / cap)                                                          */
  void* Y;                /* [M, ld], channels 0 .. n_main-1                                                       */
  int ld, n_main;
  int out_f32;            /* Y holds fp32 (else the type of X)                                                     */
  float* tail;            /* [M, tail_count] fp32: channels n_main .. n_main+tail_count-1, plus tail_bias          */
  int tail_count;
  const float* tail_bias; /* [tail_count] or NULL                                                                  */
  void* workspace;        /* NULL, or scratch of pta_wide_linear_workspace_bytes(M, N): lets bf16 launches with few
                             channels split K across workgroups                                                    */
  size_t workspace_bytes;
} pta_wide_linear_args;

size_t pta_wide_linear_workspace_bytes(int M, int N);
int pta_wide_linear(const pta_wide_linear_args* host_args, pta_stream_t stream);

/* ---- Residual streams (hyper-connections) and layer norm ---------------------------------------------------------
 * streams fp32 [rows][S][width].  One launch per sublayer boundary, one workgroup per row:
 *   1. bring the streams up to date: from the embedding (table != NULL: every stream = table[id] * embed_scale), or
 *      with the finished sublayer's output y: x_t <- sum_s mix[s][t] x_s + mult * out[t] * y  (all from the old ones);
 *   2. u = sum_s in[s] x_s  (in == NULL: the plain sum);
 *   3. h = layer_norm(u) * weight, without a bias, columns width .. h_ld-1 zero.
 * connect = {in[S], out[S], mix[S][S]} of the finished sublayer (out, mix) and `next_in` of the one that follows. */
typedef struct pta_streams_args {
  int dtype;              /* type of h, of the embedding table                                                     */
  int rows, width, S;     /* S in 1 .. 8                                                                           */
  float* streams;
  const void* table;      /* [vocab, width]                                                                        */
  int vocab;
  float embed_scale;
  const int32_t* ids;     /* id of row r: ids[r * ids_stride + (ids_index ? *ids_index : 0)]                       */
  int ids_stride;
  const int32_t* ids_index;
  int32_t* pos_out;       /* with ids_index: pos_out[r] = *ids_index (may be NULL)                                 */
  const float* y;         /* [rows, width] or NULL                                                                 */
  const float* out;       /* [S]                                                                                   */
  const float* mix;       /* [S, S], from -> to                                                                    */
  float mult;
  int write_streams;      /* whether step 1's result is stored                                                     */
  const int32_t* gather;  /* NULL, or: output row r is made from row gather[r] of streams and y                    */
  const float* next_in;   /* [S] or NULL                                                                           */
  const float* weight;    /* [width]                                                                               */
  float eps;
  void* h;                /* [rows, h_ld]                                                                          */
  int h_ld;
  float* sum_out;         /* NULL, or [rows, width]: the plain sum of the streams after step 1                     */
} pta_streams_args;

int pta_streams_norm(const pta_streams_args* host_args, pta_stream_t stream);

/* ---- Windowed attention with a distance bias ---------------------------------------------------------------------
 * score(i, j) = scale * (q_i . k_j) - slope_h * (i - j) for 0 <= i - j < window, ordinary softmax, and the concatenated
 * heads times sigmoid(gate).  q and k are RMS-normalised over the whole projection (all heads) with plain weights; the
 * VALUES ARE THE KEYS as projected, before their norm.  So the cache holds one raw row per token and key head plus one
 * fp32 factor per token (the inverse root mean square of its keys): the key norm's weight is folded into the query.
 * Cache of a layer: ring [slots][G][ring_len][Dp] (Dp = D rounded up to 8), rinv fp32 [slots][ring_len]; position p is
 * row p % ring_len, and ring_len >= window - 1 + (most rows a sequence has in one pass). */
typedef struct pta_window_attention_args {
  int dtype;
  int rows, H, G, D;
  const void* q;          /* [rows, ld], first query channel; k and gate likewise (same ld)                        */
  const void* k;
  const void* gate;
  int ld;
  const float* q_norm;    /* [H * D]                                                                               */
  const float* k_norm;    /* [G * D]                                                                               */
  float eps, scale;
  const float* slopes;    /* [H]                                                                                   */
  int window;             /* > 0                                                                                   */
  void* ring;
  float* rinv;
  int ring_len;
  const int32_t* slot;    /* [rows]                                                                                */
  const int32_t* pos;     /* [rows]                                                                                */
  float* q_scale;         /* [rows] scratch of pta_window_append                                                   */
  const int32_t* tile_row;   /* [tiles] first row of a tile: rows of one sequence, at most PTA_WINDOW_TILE          */
  const int32_t* tile_count; /* [tiles]                                                                            */
  int tiles;
  int splits;             /* decode: parts the window is cut into (1: the workgroup writes the result itself)      */
  void* workspace;        /* decode with splits > 1: pta_window_attention_workspace_bytes                          */
  size_t workspace_bytes;
  void* out;              /* [rows, out_ld]: H * D channels, the rest of out_ld zero                               */
  int out_ld;
} pta_window_attention_args;

enum { PTA_WINDOW_TILE = 128 };

size_t pta_window_attention_workspace_bytes(int rows, int H, int D, int splits);
/* every row's keys into the ring, rinv, and q_scale[r] = 1 / rms of its query projection */
int pta_window_append(const pta_window_attention_args* host_args, pta_stream_t stream);
/* rows whose keys are in the ring already (pta_window_append): bf16 on the matrix unit over tiles of rows where D <= 256,
 * else row by row */
int pta_window_attention(const pta_window_attention_args* host_args, pta_stream_t stream);
/* one row per sequence: norm, append and attention in one launch (two with splits > 1) */
int pta_window_decode(const pta_window_attention_args* host_args, pta_stream_t stream);

/* ---- Matrix memory (mLSTM) ---------------------------------------------------------------------------------------
 * Per head, with log gates i = cap tanh(z_i / cap), f = log sigmoid(cap tanh(z_f / cap)) from the fp32 pre-activations:
 *   m' = max(f + m, i);  S = exp(f + m - m') S + exp(i - m') k v^T;  n likewise with k alone;
 *   o = S^T q / (max(|n . q|, exp(-m')) + 1e-6),  q scaled by D^-1/2.
 * State of a layer, fp32: [slots][H][slices][D * PTA_MLSTM_SLICE + D + 2, up to a multiple of 4]: a head's columns of S (E of them, in slices of
 * PTA_MLSTM_SLICE, each [D][PTA_MLSTM_SLICE]), followed by that slice's own copy of n and m. */
enum { PTA_MLSTM_SLICE = 32 };

typedef struct pta_mlstm_args {
  int dtype;
  int rows, H, D, E;
  const void* q;          /* [rows, ld]: H * D channels; k likewise, v H * E                                       */
  const void* k;
  const void* v;
  int ld;
  const float* gates;     /* fp32 [rows, 2 H]: input-gate then forget-gate pre-activations, biases added           */
  float cap;
  float* state;
  const int32_t* slot;    /* [rows]                                                                                */
  const int32_t* seq_row; /* [seqs] first row of each sequence of the pass, seq_count its rows                     */
  const int32_t* seq_count;
  int seqs;
  int longest;            /* rows of the longest sequence of the pass                                              */
  int chunked;            /* bf16: work through the rows in chunks on the matrix unit where D <= 256 (else: one by one) */
  float* o;               /* fp32 [rows, H * E]                                                                    */
  void* workspace;        /* chunked: pta_mlstm_workspace_bytes (0 where the pass is not cut into segments)        */
  size_t workspace_bytes;
} pta_mlstm_args;

size_t pta_mlstm_state_floats(int H, int D, int E);   /* per slot */
size_t pta_mlstm_workspace_bytes(const pta_mlstm_args* host_args);   /* reads the sizes only */
int pta_mlstm(const pta_mlstm_args* host_args, pta_stream_t stream);

/* out = (o of each head / its root mean square) * weight * sigmoid(gate); out [rows, out_ld], the rest of a row zero */
int pta_head_norm_gate(int dtype, const float* o, const float* weight, const void* gate, int gate_ld, void* out, int out_ld,
                       int rows, int H, int E, float eps, pta_stream_t stream);

/* ---- Next-token selection over fp32 logits, and the loop's bookkeeping -------------------------------------------- */
int pta_argmax_f32(const float* logits, int32_t* ids, float* values, int rows, int n, pta_stream_t stream);
int pta_topk_f32(const float* logits, int32_t* ids, float* values, int rows, int n, int k, pta_stream_t stream);

#ifdef __cplusplus
}
#endif
#endif
