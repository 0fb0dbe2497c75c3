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
  /* main channels, in this order: sum + bias, cap, act, * mul, += Y */
  const float* bias;      /* [n_main] or NULL (of a pair: the gate's)                                              */
  const float* bias2;     /* [n_main] or NULL: the up weight's of a pair                                           */
  int act;                /* PTA_ACT_* of poptransformer_hip.h, in fp32 (single weights)                           */
  const void* mul;        /* NULL, or [M, ld] of the type of X: y = y * mul                                        */
  int accumulate;         /* Y += y (fp32 Y only)                                                                  */
} pta_wide_linear_args;

size_t pta_wide_linear_workspace_bytes(int M, int N);
int pta_wide_linear(const pta_wide_linear_args* host_args, pta_stream_t stream);
/* up to four single weights over inputs of the same shape, each with its own input and result: one launch where
 * there are few rows, or many rows and whole tiles of channels */
int pta_wide_linear_group(const pta_wide_linear_args* host_list, int count, pta_stream_t stream);

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

/* ---- One fp32 residual, sublayers in parallel: grouped RMS norm and token shift -----------------------------------
 * x fp32 [rows][width].  With n(x) = every one of `groups` equal parts of x over its own sqrt(mean square + eps):
 *   h1 = n(x) w1,  h2 = n(x) w2,  hm_t = h1_t + (h1_{t-1} - h1_t) * shift   (h1 in fp32; zeros before position 0).
 * With `table` the row is made first: x = table[id] * embed_scale + pos_table[position].
 * state fp32 [slots][width] holds h1 of a sequence's newest token.  last[r]: for the first row of a sequence in the pass
 * the row of its last token, else -1 (NULL: every row is a sequence of its own).  Positions are clamped to positions - 1. */
typedef struct pta_shift_norm_args {
  int dtype;              /* type of h1, h2, hm and of the tables                                                  */
  int rows, width, groups;
  float* x;
  const void* table;      /* [vocab, width] or NULL                                                                */
  const void* pos_table;  /* [positions, width] or NULL                                                            */
  int vocab, positions;
  float embed_scale;
  const int32_t* ids;     /* id of row r: ids[r * ids_stride + (ids_index ? *ids_index : 0)]                       */
  int ids_stride;
  const int32_t* ids_index;
  const int32_t* pos;     /* [rows]; with ids_index every row's position is *ids_index                             */
  int32_t* pos_out;       /* [rows] or NULL                                                                        */
  const int32_t* gather;  /* NULL, or: output row r is made from row gather[r]                                     */
  float eps;
  const float* w1;        /* [width]                                                                               */
  const float* w2;        /* [width], with h2                                                                      */
  const float* shift;     /* [width] or NULL                                                                       */
  float* state;
  const int32_t* slot;    /* [rows]                                                                                */
  const int32_t* last;
  void* h1;               /* [rows, h_ld], columns past width zero; h2 and hm likewise                             */
  void* h2;
  void* hm;
  int h_ld;
} pta_shift_norm_args;

int pta_shift_norm(const pta_shift_norm_args* host_args, pta_stream_t stream);

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

/* ---- Attention over latents ---------------------------------------------------------------------------------------
 * A token leaves one row in the cache: its normed latent c and one rotated key part that all heads share.  Head h has the
 * key (W_uk,h c | rotated part), the value W_uv,h c, and score(i, j) = scale * (q_i . k_j) for 0 <= i - j < window, an
 * ordinary softmax, and its result times sigmoid(gate_h), or feature by feature.  Two ways to the same numbers:
 *   absorbed (decode, short portions, fp32): q'_h = W_uk,h^T q_h meets the cached rows themselves, and W_uv,h is applied
 *     to the weighted sum of latents;
 *   over heads (prompts): keys and values of all heads are made from the cached rows (a Linear over pta_latent_gather's
 *     result) and a tile of rows works through them on the matrix unit.
 * Sizes as stored: D, P and R are the head's unrotated and rotated dimensions and the latent, each rounded up to 32 with
 * zeros, E the value size rounded up to 16.  A query head is [D | P].  Rotated features come in pairs: 2 i and 2 i + 1 are
 * turned by cos_sin[position][i], which pairs any layout's partners after a permutation of the weights' rows.
 * Cache of a layer: ring [slots][ring_len][R + P]; position p is row p % ring_len, and ring_len >= window - 1 + (most rows
 * a sequence has in one pass).  Several layers may read one cache. */
typedef struct pta_latent_args {
  int dtype;
  int rows, H, D, P, E, R;
  int q_rank, kv_rank;    /* true sizes of the two norms                                                           */
  const void* proj;       /* [rows, ld]: query latent (q_rank rounded up to 8) | latent (R) | rotated part (P)     */
  int ld;
  const float* q_norm;    /* [q_rank]                                                                              */
  const float* kv_norm;   /* [kv_rank]; NULL: the layer reads another one's cache, proj holds the query latent only */
  float eps;
  void* cq;               /* [rows, q_rank rounded up to 8]: the normed query latent                               */
  const float* cos_sin;   /* [positions][P / 2][2]                                                                 */
  int positions;
  void* ring;
  int ring_len;
  const int32_t* slot;    /* [rows]                                                                                */
  const int32_t* pos;     /* [rows]                                                                                */
  const void* q;          /* [rows, H, D + P], not rotated yet                                                     */
  const void* uk_t;       /* [H, R, D]                                                                             */
  void* q_latent;         /* [rows, H, R + P]                                                                      */
  float scale;
  int window;             /* > 0                                                                                   */
  int splits;             /* absorbed: parts a row's window is cut into, 1 .. 64                                   */
  float* part_o;          /* [rows, H, splits, R]: sums of weighted latents                                        */
  float* part_ml;         /* [rows, H, splits, 2]: their largest score and sum of weights                          */
  const void* uv;         /* [H, E, R]                                                                             */
  const float* gate;      /* [rows, H], before the sigmoid, or NULL                                                */
  const void* feature_gate; /* [rows, gate_ld], first channel of [H][E] before the sigmoid, or NULL                */
  int gate_ld;            /* a multiple of 8                                                                       */
  void* out;              /* [rows, H * E]                                                                         */
  /* over heads */
  int keys;               /* rows of the key buffers                                                               */
  const int32_t* key_slot;   /* [keys] the cache rows of pta_latent_gather                                         */
  const int32_t* key_pos;
  void* key_latent;       /* [keys, R]                                                                             */
  void* key_rot;          /* [keys, P]                                                                             */
  const void* kv;         /* [keys, H * D | H * E]                                                                 */
  const int32_t* tile_row;   /* [tiles] first row of a tile: rows of one sequence, at most PTA_LATENT_TILE          */
  const int32_t* tile_count; /* [tiles]                                                                            */
  const int32_t* tile_key;   /* [tiles] key row of the sequence's position 0 (negative where the buffer starts later) */
  int tiles;
} pta_latent_args;

enum { PTA_LATENT_TILE = 128 };

/* normed query latents; the rows' cache entries where the layer has a cache of its own */
int pta_latent_append(const pta_latent_args* host_args, pta_stream_t stream);
int pta_latent_absorb(const pta_latent_args* host_args, pta_stream_t stream);
/* every row over its part of the cache: bf16 on the matrix unit where R <= 1024 and P <= 128, else on the vector unit */
int pta_latent_rows(const pta_latent_args* host_args, pta_stream_t stream);
/* parts put together, W_uv, gate */
int pta_latent_values(const pta_latent_args* host_args, pta_stream_t stream);
int pta_latent_gather(const pta_latent_args* host_args, pta_stream_t stream);
/* whether pta_latent_tiles takes these sizes */
int pta_latent_tiles_fit(int dtype, int D, int P, int E);
int pta_latent_tiles(const pta_latent_args* host_args, pta_stream_t stream);

/* ---- Short causal convolutions -------------------------------------------------------------------------------------
 * y_t = act(sum_j weight[j] * u_{t - taps + 1 + j} + bias) channel by channel, zeros before position 0; act: silu or nothing.
 * ring [slots][taps][channels] of the rows' type keeps a sequence's newest rows, position p in row p % taps. */
typedef struct pta_conv {
  int channels, taps;     /* channels: a multiple of 8; 1 <= taps <= PTA_CONV_TILE                                 */
  const float* weight;    /* [taps][channels]                                                                      */
  const float* bias;      /* [channels] or NULL                                                                    */
  int silu;
  void* ring;             /* NULL where the struct is part of another's arguments: no convolution                  */
} pta_conv;

enum { PTA_CONV_TILE = 128 };

typedef struct pta_short_conv_args {
  int dtype;
  pta_conv c;
  const void* x;          /* [rows, ld_x]                                                                          */
  int ld_x;
  void* y;                /* [rows, ld_y]                                                                          */
  int ld_y;
  const int32_t* slot;    /* [rows]                                                                                */
  const int32_t* pos;     /* [rows]                                                                                */
  const int32_t* last;    /* [rows]: of a sequence's first row in the pass the row of its last token, else -1      */
  const int32_t* tile_row;   /* [tiles] first row of a tile: rows of one sequence, at most PTA_CONV_TILE, all of them
                                but its last that many                                                             */
  const int32_t* tile_count; /* [tiles]                                                                            */
  int tiles;
} pta_short_conv_args;

int pta_short_conv(const pta_short_conv_args* host_args, pta_stream_t stream);

/* ---- Attention over cached keys and values, by heads ---------------------------------------------------------------
 * H query heads on G key/value heads.  Query and key: RMS norm per head (plain weights), rotation of the first `rot`
 * features (pairs 2 i and 2 i + 1 turned by cos_sin[position][i]; any other pairing after a permutation of the weights'
 * rows).  The values are a projection of their own, or the keys as projected (v points at k).
 *   score(i, j) = scale * (q_i . k_j)   for j <= i with (i - j < window or j < keep) and floor(i / chunk) = floor(j / chunk)
 * less the penalty of the distance where there is one, and a softmax, whose denominator also holds exp(sink) of the head where there are sinks.  With maps = 2 every head has two
 * queries and keys [map 1 | map 2] over the same values, and its result is  o = a1 - lambda * a2,  o / sqrt(mean(o^2) + eps) *
 * (1 - diff).  Then the gates: sigmoid per head, or per feature.
 * Sizes as stored: D and E (query / key and value features) are multiples of 8, zero past `dim` and `vdim`.
 * Cache of a layer: keys (normed, rotated) [slots][G][maps][ring_len][D], values [slots][G][ring_len][E].  The first `keep`
 * positions have rows of their own; position p past them is row keep + (p - keep) % (ring_len - keep), and ring_len - keep >=
 * min(window, chunk) - 1 + (most rows a sequence has in one pass). */
typedef struct pta_head_attention_args {
  int dtype;
  int rows, H, G, maps, D, E;
  int dim, vdim;          /* true sizes                                                                            */
  const void* q;          /* [rows, ld], first query channel: [H][maps][D]                                         */
  const void* k;          /* [G][maps][D]                                                                          */
  const void* v;          /* [G][E]                                                                                */
  int ld;                 /* a multiple of 8                                                                       */
  const float* q_norm;    /* [D] or NULL: no norm                                                                  */
  const float* k_norm;    /* [D] or NULL                                                                           */
  float eps, scale;
  const float* cos_sin;   /* [positions][rot / 2][2]                                                               */
  int positions, rot;     /* rot: a multiple of 8, at most D; 0: no rotation                                       */
  int window;             /* > 0; past any position: all                                                           */
  int keep;               /* first positions that stay visible, 0: none                                            */
  int chunk;              /* 0: none (with keep = 0 only)                                                          */
  void* keys;
  void* values;
  int ring_len;
  const int32_t* slot;    /* [rows]                                                                                */
  const int32_t* pos;     /* [rows]                                                                                */
  const float* sink;      /* [H] or NULL                                                                           */
  float lambda, diff;     /* maps = 2                                                                              */
  const float* head_gate; /* [rows, H] before the sigmoid, or NULL                                                 */
  const void* gate;       /* [rows, ld], first channel of [H][E] before the sigmoid, or NULL                       */
  const int32_t* tile_row;   /* [tiles] first row of a tile: rows of one sequence, at most PTA_HEAD_TILE            */
  const int32_t* tile_count; /* [tiles]                                                                            */
  int tiles;
  int splits;             /* decode: parts the visible keys are cut into, 1 .. 64                                  */
  void* workspace;        /* decode with splits > 1: pta_head_attention_workspace_bytes                            */
  size_t workspace_bytes;
  void* out;              /* [rows, H * E]                                                                         */
  const float* far1;      /* [H] or NULL: far1 ln(1 + far2 (i - j)) is taken off the scores (keep = 0, maps = 1)   */
  const float* far2;      /* [H], not negative                                                                     */
  pta_conv conv;          /* decode: q | k | v, one behind the other, go through it first (maps = 1)               */
} pta_head_attention_args;

enum { PTA_HEAD_TILE = 128 };

size_t pta_head_attention_workspace_bytes(int rows, int H, int maps, int E, int splits);
/* every row's keys and values into the cache */
int pta_head_append(const pta_head_attention_args* host_args, pta_stream_t stream);
/* rows whose keys are in the cache already (pta_head_append): bf16 on the matrix unit over tiles of rows where D and E <= 256,
 * else row by row */
int pta_head_attention(const pta_head_attention_args* host_args, pta_stream_t stream);
/* one row per sequence: norm, rotation, append and attention in one launch (two with splits > 1) */
int pta_head_decode(const pta_head_attention_args* host_args, pta_stream_t stream);

/* ---- Residual that takes normed results, and routing ---------------------------------------------------------------
 * x fp32 [rows][width]:  x <- x + rms_norm(y) * weight  for a finished sublayer's result y, which is
 *   y[r] * (y_weight ? y_weight[r * weights_ld] : 1)  +  sum_p part_weight[r * weights_ld + p] * parts[r][p],
 * or with `table` x = table[id] * embed_scale; then h = x (what the next sublayer reads), or with final_weight the model's norm
 * of x.  With `router` the row is routed as well, by what h holds of it (pta_route_args). */
typedef struct pta_routing {
  int experts, top;       /* 1 <= top <= experts <= PTA_MAX_EXPERTS                                                */
  int shared;             /* 1: logit `experts` is a shared expert's: choice `top` of every row, weight = its sigmoid */
  float scale;
  int32_t* chosen;        /* [rows, top + shared]: largest scores first (a shared expert is number `experts`) */
  float* weights;         /* [rows, top + shared]: score * scale                                                   */
  int score;              /* PTA_SCORE_*                                                                           */
  const float* correction; /* [experts] or NULL: added to sigmoid scores for the choice, not for the weights       */
  int groups, keep;       /* equal groups of neighbouring experts (1: none); only those of the `keep` groups whose two largest
                             choice scores sum up highest can be chosen (sigmoid scores)                           */
  int share;              /* 1: a weight is the score's share of the chosen scores' sum (+ 1e-20)                  */
} pta_routing;

enum { PTA_MAX_EXPERTS = 1024 };
enum { PTA_SCORE_SOFTMAX = 0, PTA_SCORE_SIGMOID = 1 };

typedef struct pta_result_norm_args {
  int dtype;              /* type of h, of the embedding table, of the router                                      */
  int rows, width;
  float* x;
  const void* table;      /* [vocab, width] or NULL                                                                */
  int vocab;
  float embed_scale;
  const int32_t* ids;     /* id of row r: ids[r * ids_stride + (ids_index ? *ids_index : 0)]                       */
  int ids_stride;
  const int32_t* ids_index;
  int32_t* pos_out;       /* with ids_index: pos_out[r] = *ids_index (may be NULL)                                 */
  const float* y;         /* [rows, width] or NULL                                                                 */
  const float* y_weight;
  const void* parts;      /* [rows, parts_ld, width] or NULL, the first n_parts of a row                           */
  int n_parts, parts_ld;
  int part_f32;           /* fp32 parts, else of the type of h                                                     */
  const float* part_weight;
  int weights_ld;
  const float* weight;    /* [width]                                                                               */
  float eps;
  const float* final_weight; /* [width] or NULL                                                                    */
  void* h;                /* [rows, h_ld], columns past width zero                                                 */
  int h_ld;
  const void* router;     /* [experts + shared, h_ld] of the type of h, or NULL                                    */
  pta_routing routing;
} pta_result_norm_args;

int pta_result_norm(const pta_result_norm_args* host_args, pta_stream_t stream);
/* the same routing of many bf16 rows by their products with the router [experts + shared, ld] as pta_bf16_tile leaves it, ld a multiple
 * of 8 */
int pta_route_rows(const uint16_t* h, int ld, int rows, const void* router, const pta_routing* host_routing, pta_stream_t stream);
/* and of rows whose logits fp32 [rows, experts + shared] are there already */
int pta_route(const float* logits, int rows, const pta_routing* host_routing, pta_stream_t stream);

/* ---- Mixture of experts -------------------------------------------------------------------------------------------
 * Assignment a = r * choices + c is choice c of row r, done by expert chosen[a].  Two products per expert, with the epilogues
 * of pta_wide_linear's pairs between them:
 *   pta_experts with W2:    Y[a] = pair(W x_r, W2 x_r)       (X [rows, ld_x])
 *   pta_experts without:    Y[a] = W x_a                     (X [rows * choices, ld_x])
 * Weights of an expert are tiled as pta_bf16_tile leaves them (fp32: row-major), expert after expert, N a multiple of 16 (bf16).
 * Two ways: directly, every expert finding its rows itself (bf16, up to 16 rows), where the last choice may be a shared expert of
 * sizes of its own; or grouped by pta_group_experts, without it. */
typedef struct pta_expert_weights {
  const void* W;
  const void* W2;
  int K, N, n_main;       /* channels n_main .. N - 1 are padding and go nowhere; K a multiple of 8                */
  int pair;
  float limit, slope;
} pta_expert_weights;

typedef struct pta_experts_args {
  int dtype;
  int rows, experts, top, choices;   /* choices = top, or top + 1 with a shared expert                             */
  const int32_t* chosen;  /* [rows, choices]                                                                       */
  const void* X;
  int ld_x;
  pta_expert_weights routed, shared; /* shared.W NULL: no shared expert in this launch                             */
  void* Y;                /* [rows * choices, ld_y]                                                                */
  int ld_y, out_f32;
  /* grouped: pta_group_experts; NULL: directly */
  const int32_t* lists;
  int tile_rows;          /* rows of a tile of the lists, 128 or 256                                               */
} pta_experts_args;

/* int32 elements of the lists: order of the assignments (choice < top) by expert, then tiles of rows of one expert */
size_t pta_expert_lists_size(int rows, int top, int experts, int tile_rows);
int pta_group_experts(const int32_t* chosen, int rows, int top, int choices, int experts, int tile_rows, int32_t* lists, pta_stream_t stream);
int pta_experts(const pta_experts_args* host_args, pta_stream_t stream);

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

/* ---- State-space recurrence (Mamba-2) -----------------------------------------------------------------------------
 * Per head, with dt = softplus(z + dt_bias) from the fp32 pre-activations and b, c of the head's group (H / G heads share them):
 *   S = exp(-exp(a_log) dt) S + dt b x^T,   y = S^T c + skip x.
 * State of a layer, fp32: [slots][H][slices][D][PTA_SSD_SLICE], a head's columns of S (E of them) in slices.
 * With conv.ring every sequence has one row, x | b | c stand one behind the other as projected and go through the convolution first. */
enum { PTA_SSD_SLICE = 32 };

typedef struct pta_ssd_args {
  int dtype;
  int rows, H, G, D, E;   /* D (state) and E (head size): multiples of 8                                           */
  const void* x;          /* [rows, ld]: H * E channels                                                            */
  const void* b;          /* G * D                                                                                 */
  const void* c;          /* G * D                                                                                 */
  int ld;
  const float* dt;        /* fp32 [rows, H]                                                                        */
  const float* dt_bias;   /* [H]                                                                                   */
  const float* a_log;     /* [H]                                                                                   */
  const float* skip;      /* [H]                                                                                   */
  float* state;
  const int32_t* slot;    /* [rows]                                                                                */
  const int32_t* pos;     /* [rows], with conv                                                                     */
  const int32_t* seq_row; /* [seqs] first row of each sequence of the pass, seq_count its rows                     */
  const int32_t* seq_count;
  int seqs;
  int longest;            /* rows of the longest sequence of the pass                                              */
  int chunked;            /* bf16: work through the rows in chunks on the matrix unit where D <= 256 (else: one by one) */
  float* y;               /* fp32 [rows, H * E]                                                                    */
  void* workspace;        /* chunked: pta_ssd_workspace_bytes (0 where the pass is not cut into segments)          */
  size_t workspace_bytes;
  pta_conv conv;
} pta_ssd_args;

size_t pta_ssd_state_floats(int H, int D, int E);     /* per slot */
size_t pta_ssd_workspace_bytes(const pta_ssd_args* host_args);   /* reads the sizes only */
int pta_ssd(const pta_ssd_args* host_args, pta_stream_t stream);

/* out = n(y silu(z)) weight, n dividing each of `parts` equal stretches of the H * vdim columns by its own root mean square.
 * Heads are stored in E columns (vdim rounded up to 8). */
typedef struct pta_gated_norm_args {
  int dtype;
  int rows, H, E, vdim, parts;
  const float* y;         /* [rows, H * E]                                                                         */
  const void* z;          /* [rows, ld_z]                                                                          */
  int ld_z;
  const float* weight;    /* [H * E]                                                                               */
  float eps;
  void* out;              /* [rows, H * E]                                                                         */
} pta_gated_norm_args;

int pta_gated_norm(const pta_gated_norm_args* host_args, pta_stream_t stream);

/* ---- Residuals of all depths ---------------------------------------------------------------------------------------
 * history fp32 [depths][depth_stride]: the residual rows [rows][width] as the embedding (depth 0) and every layer left them.
 * One launch per end of a layer, for the newest of `depth` of them:
 *   newest += n(y) y_weight    (n: over the root mean square; where there is a y)
 *   u = sum_j weights[j] history[j]   (weights NULL with depth = 1: the row itself)
 *   next = u;  h = norm(u) norm_weight (layer norm where `centred`, else RMS norm), columns past width zero;
 * and with `router` the row is routed by what h holds (pta_route_args).  With `table` (depth = 0) u is the embedding, which is
 * also stored as history[0], and every layer's part of the token's row of side_table goes to side[layer][row]. */
typedef struct pta_depth_norm_args {
  int dtype;              /* type of h, of the tables, of the router                                               */
  int rows, width;
  float* history;
  size_t depth_stride;    /* floats                                                                                */
  int depth;
  const float* weights;   /* [depth]                                                                               */
  const float* y;         /* [rows, width] or NULL                                                                 */
  const float* y_weight;  /* [width]                                                                               */
  float* next;            /* [rows, width] or NULL                                                                 */
  int centred;
  const float* norm_weight; /* [width]                                                                             */
  float eps;              /* of both norms                                                                         */
  void* h;                /* [rows, h_ld]                                                                          */
  int h_ld;
  const void* table;      /* [vocab, width] or NULL                                                                */
  int vocab;
  float embed_scale;
  const int32_t* ids;     /* id of row r: ids[r * ids_stride + (ids_index ? *ids_index : 0)]                       */
  int ids_stride;
  const int32_t* ids_index;
  int32_t* pos_out;       /* with ids_index: pos_out[r] = *ids_index (may be NULL)                                 */
  const void* side_table; /* [vocab, side_layers, side_ld]                                                         */
  void* side;             /* [side_layers][side_stride], or NULL                                                   */
  int side_layers, side_ld; /* side_ld: a multiple of 8                                                            */
  size_t side_stride;
  const void* router;     /* [experts + shared, h_ld] of the type of h, or NULL                                    */
  pta_routing routing;
} pta_depth_norm_args;

int pta_depth_norm(const pta_depth_norm_args* host_args, pta_stream_t stream);

/* x += sum_p part_weight[r * weights_ld + p] * parts[r][p] (where there are parts), h = x, columns past width zero */
typedef struct pta_add_parts_args {
  int dtype;
  int rows, width;
  float* x;               /* [rows, width]                                                                         */
  const void* parts;      /* [rows, parts_ld, width] or NULL, the first n_parts of a row                           */
  int n_parts, parts_ld;
  int part_f32;           /* fp32 parts, else of the type of h                                                     */
  const float* part_weight;
  int weights_ld;
  void* h;                /* [rows, h_ld]                                                                          */
  int h_ld;
} pta_add_parts_args;

int pta_add_parts(const pta_add_parts_args* host_args, pta_stream_t stream);

/* ---- Next-token selection over fp32 logits, and the loop's bookkeeping -------------------------------------------- */
int pta_argmax_f32(const float* logits, int32_t* ids, float* values, int rows, int n, pta_stream_t stream);
int pta_topk_f32(const float* logits, int32_t* ids, float* values, int rows, int n, int k, pta_stream_t stream);

#ifdef __cplusplus
}
#endif
#endif
