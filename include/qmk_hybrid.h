/*
 * qmk_hybrid.h — C ABI of the hybrid route (libqmk_hybrid.so): decoders whose layers mix linear recurrences, wkv
 * time mixing and latent attention on a hyper-connected residual stream, or gated linear attention, softmax attention and
 * gated delta rules, some side by side, on a plain residual that a stretch of layers may run over several times.
 *
 * Two entry points share one layer table, one set of weights and one set of per-slot states:
 *   qmk_hybrid_decode_step   one token: ONE launch of a persistent kernel that executes an instruction tensor
 *                            (32 int32 words per instruction, one queue per workgroup), as the other routes' kernels do
 *   qmk_hybrid_prefill       a portion of 1..portion_rows tokens: one launch per fused operation of a layer
 * A portion may start anywhere; both leave the states exactly where the other expects them.
 *
 * All sizes are run-time values.  Pointers are raw DEVICE pointers owned by the caller (except `layers`, the host copy
 * of the layer table); nothing is allocated, nothing is kept after the call, launches are asynchronous on `stream`.
 *
 * Storage sizes are padded to multiples of 16 by the caller with zero weights (rows and columns), so that every row of
 * a matrix starts on a 16-byte boundary and every fourth output belongs to one lane; the true sizes enter only where a
 * mean is taken.
 */
#ifndef QMK_HYBRID_H_
#define QMK_HYBRID_H_

#include <stdint.h>

#ifdef __cplusplus
extern "C" {
#endif

#define QMK_HYBRID_ABI_VERSION 2
#define QMK_HYBRID_MAX_STREAMS 8
#define QMK_HYBRID_MAX_TAPS 16

/* element type of caches and of the activations between the prefill kernels; the decode kernel's activations are fp32 */
enum { QMK_HYBRID_BF16 = 0, QMK_HYBRID_F32 = 1 };
/* Entries of the layer table.  RGLRU, LATENT and WKV are layers on residual streams.  The others work on a plain residual:
 * GLA, ATTENTION and DELTA are mixers, each a branch of a layer run; the branches of a run follow one another in the table,
 * read the same normed input, and the first carries the run's norm and feed-forward.  JOIN replaces the residual x by
 * in_w [x; embedding]; FINAL is the model's norm.  A table holds entries of one kind only, and a plain one ends with FINAL. */
enum { QMK_MIXER_RGLRU = 0, QMK_MIXER_LATENT = 1, QMK_MIXER_WKV = 2, QMK_MIXER_GLA = 3, QMK_MIXER_ATTENTION = 4, QMK_MIXER_DELTA = 5,
       QMK_ENTRY_JOIN = 6, QMK_ENTRY_FINAL = 7 };
#define QMK_HYBRID_MAX_BRANCHES 2
/* norms of an entry; RMS: x / sqrt(mean x^2 + eps), LAYER: the same of x - mean x */
enum { QMK_NORM_RMS = 0, QMK_NORM_LAYER = 1 };
/* what a feed-forward does to its gate */
enum { QMK_ACT_GELU = 0, QMK_ACT_SILU = 1 };

/* One entry: sizes (storage sizes unless said otherwise) and pointers.  Weight matrices are bf16 [rows, columns],
 * vectors fp32.  D = storage width of the residual. */
typedef struct QmkHybridLayer {
  int32_t type;          /* QMK_MIXER_* */
  int32_t has_mlp;
  int32_t in_rows;       /* rows of in_w */
  int32_t mix_width;     /* columns of o_w: what the mixer hands to its output projection */
  int32_t heads;
  int32_t head_dim;      /* latent: unrotated part of a head; wkv: head size */
  int32_t head_dim_true; /* wkv: the head size the per-head mean is taken over */
  int32_t rot_dim;       /* latent: storage size of the rotated part */
  int32_t rot_true;      /* latent: rotated dimensions (even) */
  int32_t q_stride;      /* latent: storage of one head's query, [head_dim | rot_dim | zeros], multiple of 32 */
  int32_t v_dim;
  int32_t rank;          /* latent: storage size of the latent; wkv: storage rank of the decay's first matrix */
  int32_t rank_true;     /* latent: the size its norm's mean is taken over */
  int32_t window;        /* latent: keys a query sees, itself included */
  int32_t ring;          /* latent: rows of one slot's cache; position p lives in row p % ring */
  int32_t taps;          /* rglru: convolution taps */
  int32_t blocks;        /* rglru: blocks of the gates */
  int32_t block_dim;     /* rglru: storage size of one block; mix_width = blocks * block_dim */
  int32_t ff;            /* storage size of the feed-forward */
  float scale;           /* latent, attention: score scale */
  int32_t kv_heads;      /* attention, delta, gla: key heads; head h uses key head h / (heads / kv_heads) */
  int32_t v_true;        /* delta, gla: the value size the per-head mean is taken over */
  int32_t gate_rank;     /* delta: storage rank of the output gate */
  int32_t norm;          /* QMK_NORM_* */
  int32_t act;           /* QMK_ACT_* */
  int32_t branch;        /* plain residual: place of this entry among its run's branches */
  int32_t branches;
  int32_t prev;          /* plain residual: first entry of the run whose outputs are added to x before it is read, -1: none */
  int32_t x_from;        /* decode: the copy of x that is read (-1: the embedding) and the one that is left */
  int32_t x_to;
  int32_t proj_at;       /* decode: first element of this entry's projections (delta: in_rows, then the output gate */
  int32_t mix_at;        /* [heads * v_dim]), of what its mixer leaves and of its feed-forward's activations in a step's buffers */
  int32_t ff_at;
  float q_scale;         /* delta, gla: on the query */
  float decay_scale;     /* gla: on the logarithm of the decay */
  float out_scale;       /* a run of several branches: on the branch's normed output */
  const float* norm1;    /* [D] */
  const float* norm2;
  const uint16_t* in_w;  /* rglru: y rows, x rows; latent: q, gate, latent + rotated key; wkv: r, k, v, g, decay rank;
                            attention: q [heads][q_stride], k [kv_heads][head_dim], v [kv_heads][v_dim], gate [heads][v_dim];
                            delta: q, k [kv_heads][head_dim], v [heads][v_dim], decay rank, gate rank, steps [heads to 16];
                            gla: q, k [heads][head_dim], v, gate [heads][v_dim], decay rank; join: [D][2 D] */
  const float* in_b;     /* rglru: [in_rows], else NULL */
  const uint16_t* mid_w; /* rglru: [blocks][2 block_dim][block_dim], rows (ra_j, ri_j) interleaved;
                            latent: W_uk per head transposed [heads * rank][head_dim]; wkv, gla, delta: [heads * head_dim][rank] */
  const float* mid_b;    /* rglru: [blocks * 2 * block_dim] interleaved; wkv, delta, gla: the decay's constant [heads * head_dim] */
  const uint16_t* gate_w;/* delta: [heads * v_dim][gate_rank] */
  const uint16_t* uk_w;  /* latent: [heads * head_dim][rank] */
  const uint16_t* uv_w;  /* latent: [heads * v_dim][rank] */
  const uint16_t* o_w;   /* [D][mix_width] */
  const uint16_t* mlp_w; /* [2 ff][D], rows (gate_j, up_j) interleaved */
  const uint16_t* down_w;/* [D][ff] */
  const float* vec0;     /* rglru: -8 softplus(lam) [mix_width]; latent: weight of the latent's norm [rank];
                            wkv: weight behind the per-head norm [heads * head_dim]; delta, gla: the same [v_dim] */
  const float* vec1;     /* rglru: convolution bias [mix_width]; wkv: bonus [heads * head_dim]; delta: -exp(A_log) [heads] */
  const float* vec2;     /* rglru: convolution taps [taps][mix_width]; wkv: mixes r, k, v, g, w [5][D];
                            delta: convolution taps [taps][channels of q, k, v] */
  const float* rope_cos; /* latent, attention: [positions][rot_true / 2] */
  const float* rope_sin;
  const float* hc;       /* in1 [S], out1 [S], mix1 [S][S] ([from][to]), in2, out2, mix2 */
  const float* next1;    /* input weights of the sublayer that follows the mixer (ones behind the last one), [S] */
  const float* next2;    /* ... the feed-forward */
  const float* out_norm; /* a run of several branches: weight of the norm over the branch's output [D] */
  void* cache;           /* latent: [slots][ring][rank + rot_dim]; attention: [slots][ring][kv_heads][head_dim (key) | v_dim];
                            element type of the launch */
  float* state;          /* rglru: [slots][mix_width]; wkv: [slots][heads][head_dim (key)][head_dim (value)];
                            delta, gla: [slots][heads][head_dim][v_dim] */
  float* shift;          /* rglru: [slots][2][taps - 1][mix_width] last inputs of the convolution, oldest first;
                            delta: the same, [taps - 1][channels]; wkv: [slots][2][D] the previous token's input.  The launch reads copy `flip`, writes 1 - flip */
} QmkHybridLayer;

typedef struct QmkHybridArgs {
  uint32_t struct_size;
  uint32_t dtype;               /* QMK_HYBRID_* */
  uint32_t flags;               /* 0 */
  uint32_t spin_limit;          /* 0 = default */
  const QmkHybridLayer* layers;        /* host */
  const QmkHybridLayer* layers_device; /* the same bytes on the device */
  int32_t num_layers;
  int32_t width;                /* storage width D */
  int32_t width_true;
  int32_t streams;              /* 0: a plain residual */
  int32_t vocab;                /* tokens */
  int32_t vocab_rows;           /* storage rows of embed and head */
  int32_t slots;
  int32_t slot;
  int32_t position;             /* of the (first) token */
  int32_t max_positions;        /* rows of the rotation tables */
  int32_t flip;                 /* which copy of `shift` this launch reads */
  int32_t tokens;               /* prefill: tokens of the portion */
  int32_t num_want;             /* prefill: rows of `logits` to compute */
  int32_t portion_rows;         /* prefill: tokens the workspace was sized for */
  float eps;
  float logit_scale;
  float logit_softcap;          /* logits <- cap tanh(logits / cap); 0: none */
  int32_t reserved0;
  const uint16_t* embed;        /* bf16 [vocab_rows][D] */
  const float* final_norm;      /* [D] */
  const uint16_t* head;         /* bf16 [vocab_rows][D] */
  const int64_t* token_in;      /* prefill: [tokens]; decode: [1] */
  int64_t* token_out;           /* decode: the greedy token, or NULL */
  const int32_t* want;          /* prefill: [num_want] places in the portion */
  float* logits;                /* decode [vocab_rows]; prefill [num_want][vocab_rows] */
  float* layer_out;             /* prefill: sum of the streams behind each layer [num_layers][tokens][D], or the plain residual
                                   behind each layer run [runs][tokens][D], or NULL */
  void* workspace;              /* qmk_hybrid_decode_bytes / qmk_hybrid_prefill_bytes, 256-byte aligned, zeroed once */
  uint64_t workspace_bytes;
  /* decode only */
  const int32_t* instructions;  /* [num_queues][num_insts][32] */
  int32_t* barriers;            /* [groups][54][48], zero before the first launch; cleared by the kernel */
  int32_t num_queues;
  int32_t num_insts;
  int32_t barrier_groups;
  int32_t max_splits;           /* split-KV parts the workspace holds per head */
  uint64_t* timeline;           /* [num_queues][num_insts][8] or NULL */
  void* stream;
} QmkHybridArgs;

/* Return values are those of qmk.h (QMK_OK, QMK_ERR_*). */
int qmk_hybrid_decode_step(const QmkHybridArgs* args);
int qmk_hybrid_prefill(const QmkHybridArgs* args);
/* Workspace sizes for this layer table (the pointers in args may be NULL, sizes must be set); 0 = sizes not supported. */
uint64_t qmk_hybrid_decode_bytes(const QmkHybridArgs* args);
uint64_t qmk_hybrid_prefill_bytes(const QmkHybridArgs* args);
/* Synchronises and returns the first device-side error (0 = none); detail = workgroup, instruction, opcode, operand. */
int qmk_hybrid_status_fetch(void* stream, int32_t detail[4]);
int qmk_hybrid_max_queues(void);
int qmk_hybrid_abi_version(void);

#ifdef __cplusplus
}
#endif
#endif
