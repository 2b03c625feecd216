/*
 * cfpp_seq.h - C ABI of the sequence models of the MI355X library: prefill in portions of any size and greedy decode of
 * decoder stacks described as a list of layers (libcfpp_seq.so).
 *
 * Plain C like cfpp.h: raw device pointers, sizes, a hipStream_t passed as void*; the same status codes (cfpp.h,
 * cfpp_status): 0 success, < 0 an argument error (nothing was launched), > 0 a hipError_t.
 *
 * A layer is
 *     x <- norm1(alpha x + attention(x))
 *     x <- norm2(alpha x + feed_forward(x))            (left out with CFPP_SEQ_FF_NONE)
 * with RMS norms whose stored weight is an offset from one, and a residual stream x that is kept in fp32.
 *
 * Attention: grouped query heads (head h reads key / value head h / (heads / kv_heads)), biases on q, k and v, an RMS norm
 * over all rows of q and over all rows of k, rotary positions on the first rot_dims dimensions of every head (dimension 2i
 * paired with 2i + 1), causal and limited to chunks of `chunk` positions counted from position 0 of the sequence, a learned
 * extra term exp(sink[h]) in the softmax denominator, and values mixed with those of the first layer that mixes.
 *
 * Feed-forward: W_down relu(W_up x)^2, or `top` experts W_down (silu(W_gate x) * (W_up x)) chosen by a table indexed by the
 * token id, each weighted 1 / top, plus an always-on shared expert of the same form.
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
typedef enum cfpp_seq_ff { CFPP_SEQ_FF_NONE = 0, CFPP_SEQ_FF_RELU2 = 1, CFPP_SEQ_FF_TABLE_EXPERTS = 2 } cfpp_seq_ff;

typedef struct cfpp_seq_layer {
    /* attention */
    int32_t heads, kv_heads, dim, vdim;    /* heads % kv_heads == 0; dim, vdim <= 256 */
    int32_t chunk;                         /* positions per chunk; 0: causal only */
    int32_t rot_dims;                      /* even, <= dim; 0: no rotation */
    int32_t v_mix;                         /* 1: this layer takes part in the value mixing */
    float rot_base, scale, v_lambda;
    const void* w_qkv;                     /* T [heads*dim + kv_heads*dim + kv_heads*vdim, width]: q rows, k rows, v rows */
    const float* b_qkv;                    /* the biases in the same order */
    const float *q_norm, *k_norm;          /* [heads*dim], [kv_heads*dim] */
    const float* sink;                     /* [heads] */
    const void* w_o;                       /* T [width, heads*vdim] */
    const float* norm1;                    /* [width] */
    /* feed-forward */
    int32_t ff_kind;                       /* cfpp_seq_ff */
    int32_t ff;                            /* inner size (of one expert with CFPP_SEQ_FF_TABLE_EXPERTS) */
    int32_t experts, top, shared_ff;       /* table experts; shared_ff 0: no shared expert */
    const void *w_up, *w_down;             /* RELU2: T [ff, width], [width, ff]; experts: T [experts][2 ff, width], [experts][width, ff] */
    const void *w_shared_up, *w_shared_down;   /* T [2 shared_ff, width], [width, shared_ff] */
    const int32_t* table;                  /* [vocab, top], entries 0 .. experts - 1, those of a row differ */
    const float* norm2;                    /* [width] */
} cfpp_seq_layer;

typedef struct cfpp_seq_desc {
    int32_t dtype;                         /* cfpp_seq_dtype */
    int32_t n_layers, width, vocab;
    float eps, alpha;                      /* of every norm; of every residual sum */
    float softcap;                         /* logits <- softcap tanh(logits / softcap); 0: none */
    const cfpp_seq_layer* layers;          /* host array [n_layers] */
    const void* embed;                     /* T [vocab, width] */
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
 * tables and scratch memory.  The layer array is copied, the tensors are not. */
int cfpp_seq_create(const cfpp_seq_desc* desc, cfpp_seq** out);
int cfpp_seq_destroy(cfpp_seq* s);
/* Device bytes held by the object (caches and scratch). */
size_t cfpp_seq_bytes(const cfpp_seq* s);

/* Runs the `n` tokens at positions pos .. pos + n - 1 of the sequence in `slot`, whose positions 0 .. pos - 1 earlier calls
 * have run, and writes the logits at the places want[0 .. n_want) among them to `logits` (device fp32 [n_want, vocab]).
 * `tokens` and `want` are host arrays; want must be increasing.  One token runs through the decode kernels, more through
 * the prefill kernels.  pos == 0 starts the slot anew; a sequence cannot be wound back, since a chunk's cache rows are taken
 * over by the next chunk.  `residuals` (may be NULL): device fp32 [n_layers, n, width],
 * receives the residual stream after every layer. */
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
