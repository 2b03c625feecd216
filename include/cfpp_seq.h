/*
 * cfpp_seq.h - C ABI of the sequence models of the MI355X library: prefill in portions of any size and greedy decode of
 * decoder stacks described as a list of layers (libcfpp_seq.so).
 *
 * Plain C like cfpp.h: raw device pointers, sizes, a hipStream_t passed as void*; the same status codes (cfpp.h,
 * cfpp_status): 0 success, < 0 an argument error (nothing was launched), > 0 a hipError_t.
 *
 * Residual sum.  `streams` 0, norms after the sums:
 *     x <- norm1(alpha x + mixer(x))
 *     x <- norm2(alpha x + feed_forward(x))            (left out with CFPP_SEQ_FF_NONE)
 * `streams` s >= 1, norms in front of the sublayers and s residual streams x_1 .. x_s, all equal to the embedding at the
 * start.  Sublayer q has `in` [s], `mix` [s, s] (indexed [from, to]) and `out` [s]:
 *     y   = sublayer(norm_q(sum_a in[a] x_a))
 *     x_b <- sum_a mix[a, b] x_a + out[b] y            (all streams at once)
 * and the model's last norm reads the sum of the streams.
 * All norms are RMS norms with weight norm_offset + (stored weight); the residual streams are kept in fp32.
 *
 * Mixers.  CFPP_SEQ_MIX_GROUPED: grouped query heads (head h reads key / value head h / (heads / kv_heads)), biases on q, k
 * and v, an RMS norm over all rows of q and over all rows of k, rotary positions on the first rot_dims dimensions of every
 * head, causal and limited to chunks of `chunk` positions counted from position 0 of the sequence, and values mixed with
 * those of the first layer that mixes.
 * CFPP_SEQ_MIX_LATENT: queries of `dim` plain and rot_dims rotated dimensions per head.  Keys and values come from one latent
 * row c of kv_rank values per position (RMS norm, plain weight kv_norm): plain key W_uk c, value W_uv c, per head; the rotated
 * part of the key is one for all heads.  Cached are c and the rotated part.  kv_from >= 0: the layer reads the cache rows
 * that this earlier layer, which has its own, has made, and has none itself.  Causal.
 * Both: a learned extra term exp(sink[h]) in the softmax denominator (sink NULL: none); the latent mixer can multiply its
 * heads' outputs by sigmoid(W_g x) before W_o (gated).
 *
 * Rotary positions: pairs (2i, 2i + 1), or (i, i + rot_dims / 2) with rot_half; angle p f_i, f_i = rot_base^(-2i / rot_dims).
 * rot_factor > 0 (YaRN): f_i is blended with f_i / rot_factor between the pairs that make rot_fast and rot_slow turns over
 * rot_original positions, and cos and sin are multiplied by 0.1 ln(rot_factor) + 1.
 *
 * Feed-forward: W_down relu(W_up x)^2; or W_down (silu(W_gate x) * (W_up x)) with optional biases; or `top` experts of the
 * latter form without biases chosen by a table indexed by the token id, each weighted 1 / top, plus an always-on shared
 * expert.
 *
 * Tensors.  `dtype` is the element type T of the matrices, of the caches and of the matrix products' inputs; vectors are
 * fp32.  Every matrix is [rows, K] with the rows padded with zeros to a multiple of CFPP_SEQ_ROW_BYTES bytes (row pitch =
 * cfpp_seq_row_pitch(K, dtype)).  Gate and up matrices are one matrix with interleaved rows: row 2j = gate row j, row
 * 2j + 1 = up row j.  All pointers are device pointers, 16-byte aligned, and stay valid for the life of the model object.
 */
#ifndef CFPP_SEQ_H
#define CFPP_SEQ_H

#include <stddef.h>
#include <stdint.h>

#include "cfpp.h"

#ifdef __cplusplus
extern "C" {
#endif

#define CFPP_SEQ_ROW_BYTES 128

typedef enum cfpp_seq_dtype { CFPP_SEQ_BF16 = 0, CFPP_SEQ_F32 = 1 } cfpp_seq_dtype;
typedef enum cfpp_seq_ff { CFPP_SEQ_FF_NONE = 0, CFPP_SEQ_FF_RELU2 = 1, CFPP_SEQ_FF_TABLE_EXPERTS = 2, CFPP_SEQ_FF_GATED = 3 } cfpp_seq_ff;
typedef enum cfpp_seq_mixer { CFPP_SEQ_MIX_GROUPED = 0, CFPP_SEQ_MIX_LATENT = 1 } cfpp_seq_mixer;

#define CFPP_SEQ_MAX_STREAMS 8

/* The connections of a sublayer with the residual streams: fp32 device pointers. */
typedef struct cfpp_seq_streams {
    const float* in;                       /* [streams] */
    const float* mix;                      /* [streams, streams], indexed [from, to] */
    const float* out;                      /* [streams] */
} cfpp_seq_streams;

typedef struct cfpp_seq_layer {
    /* mixer */
    int32_t mixer;                         /* cfpp_seq_mixer */
    int32_t heads, kv_heads;               /* grouped: heads % kv_heads == 0; latent: kv_heads is not used */
    int32_t dim, vdim;                     /* per head, <= 256; latent: dim plain dimensions, dim + rot_dims <= 256 */
    int32_t chunk;                         /* grouped: positions per chunk; 0: causal only */
    int32_t rot_dims;                      /* even; grouped: of the dim, latent: beside them, <= 128; 0: no rotation */
    int32_t rot_half;                      /* pairs (i, i + rot_dims / 2) */
    int32_t v_mix;                         /* grouped: this layer takes part in the value mixing */
    int32_t kv_rank, kv_from, gated;       /* latent: kv_rank <= 512, kv_from -1: own cache rows */
    float scale, v_lambda;
    double rot_base;
    double rot_factor, rot_original, rot_fast, rot_slow;   /* rot_factor 0: no scaling of the angles */
    const void* w_qkv;                     /* T [rows, width]; grouped: heads*dim q rows, kv_heads*dim k rows, kv_heads*vdim v rows;
                                              latent: heads*(dim + rot_dims) q rows (head by head, plain part first), unless
                                              kv_from >= 0: kv_rank + rot_dims rows of the cached parts, if gated: heads*vdim rows */
    const float* b_qkv;                    /* grouped: the biases in the same order */
    const float *q_norm, *k_norm;          /* grouped: [heads*dim], [kv_heads*dim] */
    const float* kv_norm;                  /* latent, unless kv_from >= 0: [kv_rank] */
    const void* w_ukv;                     /* latent: T [heads*dim + heads*vdim, kv_rank]: W_uk rows, then W_uv rows */
    const float* sink;                     /* [heads] or NULL */
    const void* w_o;                       /* T [width, heads*vdim] */
    const float* norm1;                    /* [width] */
    cfpp_seq_streams hc1;                  /* streams >= 1 */
    /* feed-forward */
    int32_t ff_kind;                       /* cfpp_seq_ff */
    int32_t ff;                            /* inner size (of one expert with CFPP_SEQ_FF_TABLE_EXPERTS) */
    int32_t experts, top, shared_ff;       /* table experts; shared_ff 0: no shared expert */
    const void *w_up, *w_down;             /* RELU2: T [ff, width], [width, ff]; GATED: T [2 ff, width], [width, ff];
                                              experts: T [experts][2 ff, width], [experts][width, ff] */
    const float *b_up, *b_down;            /* GATED: biases in the row order of the matrices, or NULL */
    const void *w_shared_up, *w_shared_down;   /* T [2 shared_ff, width], [width, shared_ff] */
    const int32_t* table;                  /* [vocab, top], entries 0 .. experts - 1, those of a row differ */
    const float* norm2;                    /* [width] */
    cfpp_seq_streams hc2;                  /* streams >= 1 */
} cfpp_seq_layer;

typedef struct cfpp_seq_desc {
    int32_t dtype;                         /* cfpp_seq_dtype */
    int32_t n_layers, width, vocab;
    int32_t streams;                       /* residual streams with norms in front; 0: norms after the sums */
    int32_t positions;                     /* rows of `pos` */
    float eps, alpha;                      /* of every norm; of every residual sum (streams 0) */
    float norm_offset;                     /* norm weight = norm_offset + stored weight (not kv_norm, q_norm, k_norm) */
    float logit_scale, softcap;            /* logits <- cap(logit_scale * logits), cap(z) = softcap tanh(z / softcap); softcap 0: none */
    const cfpp_seq_layer* layers;          /* host array [n_layers] */
    const void* embed;                     /* T [vocab, width] */
    const void* pos;                       /* T [positions, width], added to the embedding; NULL: none (streams >= 1 only) */
    const float* final_norm;               /* [width] */
    const void* head;                      /* T [vocab, width] */
    int32_t slots;                         /* sequences that can hold cache at a time */
    int32_t capacity;                      /* positions per sequence */
    int32_t max_portion;                   /* prompt tokens per pass; longer inputs are cut into passes of this size */
} cfpp_seq_desc;

typedef struct cfpp_seq cfpp_seq;          /* opaque */

/* Bytes from one row of a T matrix with K columns to the next. */
size_t cfpp_seq_row_pitch(int32_t K, int32_t dtype);
const char* cfpp_seq_version(void);

/* Allocates the caches ([slots] x the rows a layer can see: min(chunk, capacity), or capacity without chunks), rotary
 * tables and scratch memory (latent mixers: keys and values of all heads for one sequence of `capacity` positions).  The layer array is copied, the tensors are not. */
int cfpp_seq_create(const cfpp_seq_desc* desc, cfpp_seq** out);
int cfpp_seq_destroy(cfpp_seq* s);
/* Device bytes held by the object (caches and scratch). */
size_t cfpp_seq_bytes(const cfpp_seq* s);

/* Runs the `n` tokens at positions pos .. pos + n - 1 of the sequence in `slot`, whose positions 0 .. pos - 1 earlier calls
 * have run, and writes the logits at the places want[0 .. n_want) among them to `logits` (device fp32 [n_want, vocab]).
 * `tokens` and `want` are host arrays; want must be increasing.  One token runs through the decode kernels, more through
 * the prefill kernels.  pos == 0 starts the slot anew; a sequence cannot be wound back, since a chunk's cache rows are taken
 * over by the next chunk.  `residuals` (may be NULL): device fp32 [n_layers, n, width],
 * receives the residual stream (the sum of the streams) after every layer. */
int cfpp_seq_forward(cfpp_seq* s, int32_t slot, const int32_t* tokens, int32_t n, int32_t pos, const int32_t* want,
                     int32_t n_want, float* logits, float* residuals, void* stream);

/* Greedy decode on the device: sets the (token, position) the next step starts from ... */
int cfpp_seq_set_state(cfpp_seq* s, int32_t slot, int32_t token, int32_t pos, void* stream);
/* ... runs n steps, each consuming the token, writing the logits, picking the next token (lowest index of the largest
 * logit) and storing it as the next step's: eagerly, or replaying one captured hipGraph.  CFPP_ERR_SEQ if a step would go
 * past the capacity. */
int cfpp_seq_steps(cfpp_seq* s, int32_t n, void* stream);
int cfpp_seq_graph_steps(cfpp_seq* s, int32_t n, void* stream);
/* Kernel launches of one decode step. */
int cfpp_seq_launches_per_step(const cfpp_seq* s);

/* Device pointers, to read: logits fp32 [vocab] of the last step, state int32[4] = {token, position, steps since
 * set_state, slot}, the tokens picked since set_state. */
int cfpp_seq_buffers(cfpp_seq* s, float** logits, int32_t** state, int32_t** history, int32_t* history_capacity);

#ifdef __cplusplus
}
#endif
#endif /* CFPP_SEQ_H */
