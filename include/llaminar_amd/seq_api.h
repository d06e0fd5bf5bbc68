/* C ABI of the operators behind sequence models with plain (bf16) weights: linear layers,
 * norms, routed expert feed-forwards, latent and grouped-query attention, matrix-memory and
 * delta-rule recurrences, for portions of prompts and for decoding.
 *
 * Conventions are those of ql_api.h: d_* is device memory, a call only enqueues work on
 * `stream` for `device_id`, returns false and records a message (llam_ql_last_error) on bad
 * arguments or a failed launch, allocates nothing and synchronises nothing.
 *
 * `dtype` chooses the number format of activations, caches and matrix operands:
 * LLAM_SEQ_BF16 (16-bit operands, 32-bit sums) or LLAM_SEQ_F32 (32-bit throughout, true
 * 32-bit products).  "elem" below is that format.  Residual stream, projection outputs, norms,
 * scores, router logits and recurrent state are 32-bit in both.
 *
 * Weights are bf16, N x K, in tiles: rows padded with zeros to a multiple of 16, columns to a
 * multiple of 64, then [N/16][K/32][g = 0..3][r = 0..15][8]: element (row, col) at tile row/16,
 * step col/32, g = (col % 32) / 8, r = row % 16, last index col % 8.  A 16-row step is one
 * contiguous kilobyte, the order in which the matrix unit takes it. */
#ifndef LLAMINAR_AMD_SEQ_API_H
#define LLAMINAR_AMD_SEQ_API_H

#include <stdbool.h>
#include <stddef.h>
#include <stdint.h>

#ifdef __cplusplus
extern "C" {
#endif

enum { LLAM_SEQ_BF16 = 0, LLAM_SEQ_F32 = 1 };

/* What a linear layer does with its product y [M x N]. */
enum
{
    LLAM_SEQ_OUT_F32 = 0,  /* fp32 y (+ bias), row stride ldy                                     */
    LLAM_SEQ_OUT_ADD = 1,  /* fp32 y added to what is there (the residual stream)                 */
    LLAM_SEQ_OUT_ELEM = 2, /* elem y                                                              */
    LLAM_SEQ_OUT_GATED = 3, /* elem gelu_tanh(gate) * up, N/2 columns: 16-row tiles of W alternate
                               gate, up                                                           */
    LLAM_SEQ_OUT_RELU2 = 4, /* elem max(y, 0)^2                                                   */
    LLAM_SEQ_OUT_GATED_CLAMP = 5 /* as GATED, with g = min(gate, limit), u = up within +-limit:
                                    g sigmoid(1.702 g) (u + 1)                                    */
};

/* Y = A W^T, `batch` times with the given strides (elements; w_stride counts weights).
 * A: elem [M][lda].  With d_norm set (M <= 16, batch 1) d_a is fp32 [M][lda] instead and every
 * row is RMS-normed first: x / sqrt(mean over k_real of x^2 + eps) * d_norm; d_norm has K values,
 * those from k_real on zero.  d_h_out, if set, receives the normed rows, elem [M][K].
 * N a multiple of 16, K of 64, rows 16-byte aligned. */
typedef struct
{
    const void *d_a;
    const void *d_w;
    void *d_y;
    const float *d_bias;
    const float *d_norm;
    void *d_h_out;
    float eps;
    int k_real;
    int M, N, K;
    int lda, ldy;
    int out;
    int batch;
    long a_stride, w_stride, y_stride;
    float limit; /* of LLAM_SEQ_OUT_GATED_CLAMP */
} llam_seq_linear_args;
bool llam_seq_linear(const llam_seq_linear_args *a, int dtype, int device_id, void *stream);

/* Two linear layers over the same M rows with the same K and nothing in common otherwise (the two
 * branches of a parallel layer), unbatched: up to 16 rows in one launch.  Both have d_norm or none has. */
bool llam_seq_linear_pair(const llam_seq_linear_args *a, const llam_seq_linear_args *b, int dtype, int device_id,
                          void *stream);

/* Token embedding: fp32 rows [M][ldx], scale times the id's row of a bf16 table [vocab][width]; columns
 * from width to ldx and rows of ids outside [0, vocab) are zero.
 * With d_pairs, a bf16 table [buckets + 1][width], row (previous id * mul_prev + id * mul_cur) mod
 * buckets is added, or row `buckets` where the sequence begins.  The previous id is that of the row
 * before, if it belongs to the same slot, else d_history[slot][position - 1]; every row leaves its id in
 * d_history[slot][position] ([slots][cap]).  d_row_slot / d_row_pos per row. */
typedef struct
{
    const void *d_table;
    int vocab, width;
    float scale;
    const void *d_pairs;
    int buckets;
    long mul_prev, mul_cur;
    const int32_t *d_row_slot, *d_row_pos;
    int32_t *d_history;
    int cap;
} llam_seq_embed_args;
bool llam_seq_embed(const llam_seq_embed_args *a, const int32_t *d_ids, float *d_x, int M, int ldx, int device_id,
                    void *stream);

/* elem y[m] = RMS norm of fp32 x[d_rows ? d_rows[m] : m], as in llam_seq_linear; K columns. */
bool llam_seq_rmsnorm(const float *d_x, int ldx, const int32_t *d_rows, const float *d_norm, float eps, int k_real,
                      void *d_y, int M, int K, int dtype, int device_id, void *stream);

/* Two norms of the same rows: y_a and y_b, elem [M][K], with weights d_norm_a and d_norm_b. */
bool llam_seq_rmsnorm_pair(const float *d_x, int ldx, const float *d_norm_a, const float *d_norm_b, float eps, int k_real,
                           void *d_ya, void *d_yb, int M, int K, int dtype, int device_id, void *stream);

/* Entries of a step: entry e brings d_ntok[e] tokens of the sequence in slot d_slot[e], rows
 * d_row0[e].. of the step, at positions d_pos[e].. of the sequence.  Device memory. */
typedef struct
{
    const int32_t *d_row0, *d_ntok, *d_slot, *d_pos;
} llam_seq_entries;

/* Latent rows into the cache: cache[slot][pos] = elem RMS norm of x's columns; one row per token,
 * d_row_slot / d_row_pos per row.  Cache: elem [slots][cap][rank], rank a multiple of 64 (the
 * padding zero); positions outside [0, cap) are not written. */
bool llam_seq_latent_append(const float *d_x, int ldx, const float *d_norm, float eps, int k_real,
                            const int32_t *d_row_slot, const int32_t *d_row_pos, void *d_cache, int M, int rank,
                            int cap, int dtype, int device_id, void *stream);

/* Causal softmax attention of latent queries over a latent cache that is key and value at once:
 *   o[row][h] = sum_p softmax_p(scale * q[row][h] . c[p]) c[p],  p <= the row's position.
 * q, o: elem [rows][heads][rank]; entries first .. first + n - 1 of `e`, each of at most max_ntok
 * tokens whose last position is below max_len (host bounds; max_len <= cap).
 * d_scratch: llam_seq_latent_scratch_floats floats. */
size_t llam_seq_latent_scratch_floats(int max_rows, int slots, int heads, int rank, int cap);
bool llam_seq_latent_attention(const void *d_q, const void *d_cache, const llam_seq_entries *e, int first, int n,
                               int max_ntok, int max_len, int heads, int rank, int cap, float scale, void *d_o,
                               float *d_scratch, size_t scratch_floats, int dtype, int device_id, void *stream);

/* Matrix-memory recurrence (per head a dim x vdim memory S, a vector n and a running maximum m):
 *   i = cap tanh(i_raw / cap), f = logsigmoid(cap tanh(f_raw / cap)), m' = max(f + m, i)
 *   S = e^(f + m - m') S + e^(i - m') k v^T,  n likewise with k,  m = m'
 *   o = S^T q / (max(|n . q|, e^-m) + 1e-6),  q scaled by q_scale
 * followed by y = o / rms(o) * norm * sigmoid(g) (the mean over vdim_real).
 * d_proj: fp32 rows of ldp holding q [heads][dim], k [heads][dim], v [heads][vdim],
 * g [heads][vdim], i_raw [heads], f_raw [heads]; dim and vdim multiples of 64, paddings zero.
 * d_gate_bias: [2][heads], of i then f.  d_norm: [heads][vdim].
 * State, fp32: d_state [slots][heads][dim][vdim + 16] (column vdim is n), d_m [slots][heads];
 * a sequence at position 0 starts from zeros whatever they hold.  y: elem, rows of ldy, [heads][vdim]. */
typedef struct
{
    const float *d_proj;
    int ldp;
    const float *d_gate_bias;
    const float *d_norm;
    float *d_state;
    float *d_m;
    void *d_y;
    int ldy;
    int heads, dim, vdim, vdim_real;
    float q_scale, gate_cap, eps;
} llam_seq_memory_args;
size_t llam_seq_memory_scratch_bytes(int max_rows, int heads, int dim, int vdim);
/* one token per entry, entries first .. first + n - 1 */
bool llam_seq_memory_decode(const llam_seq_memory_args *a, const llam_seq_entries *e, int first, int n,
                            void *d_scratch, size_t scratch_bytes, int dtype, int device_id, void *stream);
/* one entry of ntok tokens, in chunks */
bool llam_seq_memory_prefill(const llam_seq_memory_args *a, const llam_seq_entries *e, int entry, int ntok,
                             void *d_scratch, size_t scratch_bytes, int dtype, int device_id, void *stream);

/* Grouped-query attention with rotary positions.  Query head h reads key/value head h / (heads / kv_heads).
 * Caches: elem, k [slots][kv_heads][ring][dim], v [slots][kv_heads][ring][vdim]; position p lies in row
 * p mod ring.  dim and vdim are 64, 128 or 256 (paddings zero), ring a multiple of 128.
 * chunk > 0: position i sees j <= i of its own chunk only, i / chunk == j / chunk; 0: every j <= i. */
typedef struct
{
    int heads, kv_heads, dim, vdim;
    int ring, chunk;
    float scale;
    void *d_k, *d_v;
} llam_seq_attention_args;

/* Rotary positions and the cache: d_proj, fp32 rows of ldp holding q [heads][dim] and, with append, k
 * [kv_heads][dim] and v [kv_heads][vdim].  In every q and k head, dimension i turns with dimension
 * i + rot_dims / 2 (i < rot_dims / 2) by position * 2 pi * d_turns[i]; the others stay.  q goes to d_q, elem
 * [M][heads][dim], k and v into the cache rows of d_row_slot / d_row_pos. */
bool llam_seq_rotary(const llam_seq_attention_args *a, const float *d_proj, int ldp, bool append, const double *d_turns,
                     int rot_dims, const int32_t *d_row_slot, const int32_t *d_row_pos, void *d_q, int M, int dtype,
                     int device_id, void *stream);

/* o[row][h] = sum_j softmax_j(scale q[row][h] . k[j]) v[j] for the tokens of entries first .. first + n - 1,
 * each of at most max_ntok tokens whose last position is below max_len (host bounds); the keys in sight of
 * an entry's first token and the entry itself must lie within `ring` positions.  q as llam_seq_rotary leaves it, o: elem, rows of
 * ldo, [heads][vdim].  d_scratch: llam_seq_attention_scratch_floats floats. */
size_t llam_seq_attention_scratch_floats(int vdim);
bool llam_seq_attention(const llam_seq_attention_args *a, const void *d_q, const llam_seq_entries *e, int first, int n,
                        int max_ntok, int max_len, void *d_o, int ldo, float *d_scratch, size_t scratch_floats, int dtype,
                        int device_id, void *stream);

/* Gated delta rule (per head a dim x vdim state S; heads / kv_heads heads share q and k):
 *   q, k, v pass a causal convolution over `taps` tokens per channel and silu; q and k become unit vectors
 *   (x / sqrt(sum x^2 + 1e-6)), q times dim_real^-1/2
 *   beta = sigmoid(b), decay = exp(-exp(a_log) softplus(a + dt_bias))
 *   S = decay S;  u = beta (v - S^T k);  S = S + k u^T;  o = S^T q
 * followed by y = o / rms(o) * norm * silu(g) (the mean over vdim_real).
 * d_proj: fp32 rows of ldp holding q [kv_heads][dim], k [kv_heads][dim], v [heads][vdim], g [heads][vdim],
 * b [heads], a [heads]; dim (up to 256) and vdim multiples of 64, paddings zero.  d_conv: [taps][channels]
 * of q, k and v as they lie in the row, the last tap for the current token.  d_norm: [vdim].
 * State, fp32: d_state [slots][heads][dim][vdim], d_recent [slots][taps][channels] (inputs of the convolution,
 * position p in row p mod taps); a sequence at position 0 starts from zeros whatever they hold.
 * y: elem, rows of ldy, [heads][vdim]. */
typedef struct
{
    const float *d_proj;
    int ldp;
    const float *d_conv, *d_a_log, *d_dt_bias, *d_norm;
    float *d_state, *d_recent;
    void *d_y;
    int ldy;
    int heads, kv_heads, dim, vdim, dim_real, vdim_real, taps;
    float eps;
} llam_seq_delta_args;
size_t llam_seq_delta_scratch_bytes(int max_rows, int heads, int kv_heads, int dim, int vdim);
/* one token per entry, entries first .. first + n - 1 */
bool llam_seq_delta_decode(const llam_seq_delta_args *a, const llam_seq_entries *e, int first, int n, int dtype,
                           int device_id, void *stream);
/* one entry of ntok tokens, in chunks */
bool llam_seq_delta_prefill(const llam_seq_delta_args *a, const llam_seq_entries *e, int entry, int ntok, void *d_scratch,
                            size_t scratch_bytes, int dtype, int device_id, void *stream);

/* Routed experts.  logits: fp32 [M][ldz], column e < experts of expert e, column `experts` the
 * logit of the shared expert's gate where there is one.  Expert e's matrices: d_up + e *
 * up_stride weights (ff x K) and d_down + e * down_stride (N x ff); shared_ff = 0: no shared
 * expert.  x [M][ldx] (fp32) receives the added outputs, N columns.
 * h: elem [M][K], the normed input. */
typedef struct
{
    const float *d_logits;
    int ldz;
    const void *d_up, *d_down;
    const void *d_shared_up, *d_shared_down;
    long up_stride, down_stride;
    int experts, top, ff, shared_ff, K, N;
    const void *d_h;
    float *d_x;
    int ldx;
} llam_seq_experts_args;
size_t llam_seq_experts_scratch_bytes(int max_rows, int experts, int top, int ff, int shared_ff, int N);
bool llam_seq_experts(const llam_seq_experts_args *a, int M, void *d_scratch, size_t scratch_bytes, int dtype,
                      int device_id, void *stream);

/* d_out[*d_count * n + b] = d_ids[b], then *d_count += 1: the tokens of replayed decode steps in
 * order; nothing is written once *d_count has reached max_count. */
bool llam_seq_record(const int32_t *d_ids, int n, int32_t *d_out, int32_t *d_count, int max_count, int device_id,
                     void *stream);

#ifdef __cplusplus
}
#endif
#endif
