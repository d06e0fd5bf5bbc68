/* Host-side driver of decoder-only models whose layers are chosen one by one: each layer has a
 * token mixer (latent or grouped-query attention, a matrix-memory or a delta-rule recurrence) and a
 * feed-forward (gated, routed experts, or none), pre-norm, over plain bf16 weights.  C ABI over an opaque handle, exported by
 * libllaminar_seq.so together with the operators of seq_api.h, which do all the arithmetic.
 *
 *   x = embed_scale embed[ids] (+ a row per pair of neighbouring ids)
 *   per layer:  x += mixer(rms(x) * norm1);  x += ffn(rms(x) * norm2)
 *   or, for a parallel layer:  x += mixer(rms(x) * norm1) + ffn(rms(x) * norm2), both of the same x
 *   logits = head (rms(x) * final_norm)
 *
 * The handle owns the sequences' state: `slots` sequences of up to `cap` tokens, per latent layer
 * a cache [slots][cap][rank], per grouped-query attention layer a ring of keys and values, long enough for
 * what the masks of the layers that read it let them see (a layer with kv_from reads that layer's), per memory
 * or delta layer fp32 state, and the ids themselves where pairs of them are embedded.
 * A sequence starts afresh when an entry names its slot with position 0; nothing has to be cleared.
 *
 * llam_seqm_forward runs one step: any mixture of portions of prompts and single tokens, at most
 * max_rows tokens together.  llam_seqm_decode generates greedily, one token per sequence and step,
 * the tokens staying on the device and the steps replayed as HIP graphs.
 *
 * Functions return false (NULL) on error and keep the reason for llam_seqm_last_error(). */
#ifndef LLAMINAR_AMD_SEQUENCE_MODEL_H
#define LLAMINAR_AMD_SEQUENCE_MODEL_H

#include <stdbool.h>
#include <stddef.h>
#include <stdint.h>

#ifdef __cplusplus
extern "C" {
#endif

enum
{
    LLAM_MIXER_LATENT_ATTENTION = 1,
    LLAM_MIXER_MATRIX_MEMORY = 2,
    LLAM_MIXER_ATTENTION = 3, /* grouped-query, rotary */
    LLAM_MIXER_DELTA = 4
};
enum { LLAM_FFN_NONE = 0, LLAM_FFN_GATED = 1, LLAM_FFN_EXPERTS = 2, LLAM_FFN_GATED_CLAMP = 3 };

typedef struct
{
    int width, vocab, n_layers;
    int slots, cap, max_rows;
    int dtype; /* LLAM_SEQ_BF16 or LLAM_SEQ_F32 */
    float eps;
    int device_id;
} llam_seqm_config;

/* P(n) = n rounded up to a multiple of 64, A(n) to 64, 128 or 256, H = heads, G = kv_heads.  Matrices in the tiles of seq_api.h,
 * [rows x columns] padded with zeros; per-head blocks are padded per head.  Vectors fp32, padded
 * with zeros like the columns they belong to.  All device memory, owned by the caller. */
typedef struct
{
    int mixer;
    int heads, dim, vdim;
    const float *norm1; /* [P(width)] */
    /* latent attention: [P(q_rank) (+ P(kv_rank)) x P(width)]: query latent, then key/value latent
     * (absent with kv_from >= 0).
     * matrix memory: [2 H P(dim) + 2 H P(vdim) + 2 H, rounded up to 16, x P(width)]: q, k, v, output
     * gate, input gate, forget gate
     * attention: [H A(dim) (+ G A(dim) + G A(vdim)), x P(width)]: q (k, v absent with kv_from >= 0)
     * delta: [2 G P(dim) + 2 H P(vdim) + 2 H, rounded up to 16, x P(width)]: q, k, v, output gate, b, a */
    const void *w_in;
    /* [P(width) x H P(vdim)], attention: [P(width) x H A(vdim)]; of a parallel layer with a feed-forward
     * followed by that one's down projection, [P(width) x (H P(vdim) + P(ff))] */
    const void *w_out;
    /* latent attention */
    int q_rank, kv_rank, kv_from; /* kv_from: the layer whose cache is read, or -1 */
    float scale;
    const float *q_norm, *kv_norm; /* [P(q_rank)], [P(kv_rank)] */
    const void *w_uq;              /* [H P(dim) x P(q_rank)] */
    const void *w_uk_t;            /* H matrices [P(kv_rank) x P(dim)], transposed per head */
    const void *w_uv;              /* H matrices [P(vdim) x P(kv_rank)] */
    /* matrix memory */
    float gate_cap;
    const float *gate_bias; /* [2][H]: input gate, forget gate */
    const float *head_norm; /* [H][P(vdim)]; delta: [P(vdim)] */
    /* attention, delta */
    int kv_heads;
    /* attention; turns: [rot_dims / 2], revolutions per position; chunk 0: no mask */
    int rot_dims, chunk;
    const double *turns;
    /* delta; conv: [taps][2 G P(dim) + H P(vdim)]; a_log, dt_bias: [H] */
    int taps;
    const float *conv, *a_log, *dt_bias;
    /* feed-forward */
    int parallel; /* with gated feed-forwards; w_down is then part of w_out */
    int ffn;
    const float *norm2;
    float limit;          /* gated with clamps */
    int ff;               /* gated: its width; experts: an expert's */
    const void *w_up;     /* gated: [2 P(ff) x P(width)], 16-row tiles of gate and up alternating;
                             experts: `experts` matrices [P(ff) x P(width)] */
    const void *w_down;   /* [P(width) x P(ff)], for experts `experts` of them */
    int experts, top, shared_ff; /* shared_ff 0: no shared expert */
    const void *w_router;        /* [experts (+ 1 with a shared expert: its gate), rounded up to 16, x P(width)] */
    const float *router_bias;    /* as many values as w_router has rows */
    const void *w_shared_up, *w_shared_down; /* [P(shared_ff) x P(width)], [P(width) x P(shared_ff)] */
} llam_seqm_layer;

typedef struct
{
    const void *embed;       /* bf16 [vocab][width], row-major */
    const float *final_norm; /* [P(width)] */
    const void *head;        /* [vocab rounded up to 16 x P(width)] */
    float embed_scale;
    const void *pairs; /* bf16 [buckets + 1][width], or NULL; see llam_seq_embed */
    int buckets;
    long mul_prev, mul_cur;
} llam_seqm_globals;

void *llam_seqm_create(const llam_seqm_config *cfg);
void llam_seqm_destroy(void *model);
/* Device copy of host data, owned by the handle. */
void *llam_seqm_upload(void *model, const void *h_data, size_t bytes);
bool llam_seqm_set_layer(void *model, int layer, const llam_seqm_layer *w);
/* After the last layer: allocates caches, state and buffers. */
bool llam_seqm_set_globals(void *model, const llam_seqm_globals *g);

/* One step.  Entry e: h_ntok[e] tokens for slot h_slot[e] from position h_pos[e] on; h_ids holds
 * the entries' tokens one after the other; a slot appears at most once.  h_want: rows (places among
 * all tokens of the step) whose logits go to h_logits [n_want][vocab] (may be NULL) and whose
 * largest logit's index goes to h_best [n_want] (may be NULL).  Synchronous. */
bool llam_seqm_forward(void *model, int n, const int32_t *h_slot, const int32_t *h_pos, const int32_t *h_ntok,
                       const int32_t *h_ids, int n_want, const int32_t *h_want, float *h_logits, int32_t *h_best);

/* `steps` greedy tokens for n sequences: sequence b in slot h_slot[b] gets token h_ids[b] at
 * position h_pos[b] and continues with its own choices, h_out [steps][n].  h_ms, if set, receives
 * the duration of the steps on the device in milliseconds.  Synchronous. */
bool llam_seqm_decode(void *model, int n, const int32_t *h_slot, const int32_t *h_pos, const int32_t *h_ids, int steps,
                      int32_t *h_out, float *h_ms);

/* The residual stream after every layer of the following llam_seqm_forward calls is copied to
 * h_trace [n_layers][rows][width] (for inspection; NULL ends it). */
bool llam_seqm_trace(void *model, float *h_trace);

/* Bytes of device memory of caches and state per sequence, and of everything the handle owns. */
size_t llam_seqm_slot_bytes(void *model);
size_t llam_seqm_device_bytes(void *model);

const char *llam_seqm_last_error(void);

#ifdef __cplusplus
}
#endif
#endif
