/*
 * qmk_hybrid.h — C ABI of the hybrid route (libqmk_hybrid.so): decoders whose layers mix linear recurrences, wkv
 * time mixing and latent attention on a hyper-connected residual stream.
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

#define QMK_HYBRID_ABI_VERSION 1
#define QMK_HYBRID_MAX_STREAMS 8
#define QMK_HYBRID_MAX_TAPS 16

/* element type of caches and of the activations between the prefill kernels; the decode kernel's activations are fp32 */
enum { QMK_HYBRID_BF16 = 0, QMK_HYBRID_F32 = 1 };
/* mixers */
enum { QMK_MIXER_RGLRU = 0, QMK_MIXER_LATENT = 1, QMK_MIXER_WKV = 2 };

/* One layer: sizes (storage sizes unless said otherwise) and pointers.  Weight matrices are bf16 [rows, columns],
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
  float scale;           /* latent: score scale */
  const float* norm1;    /* [D] */
  const float* norm2;
  const uint16_t* in_w;  /* rglru: y rows, x rows; latent: q, gate, latent + rotated key; wkv: r, k, v, g, decay rank */
  const float* in_b;     /* rglru: [in_rows], else NULL */
  const uint16_t* mid_w; /* rglru: [blocks][2 block_dim][block_dim], rows (ra_j, ri_j) interleaved;
                            latent: W_uk per head transposed [heads * rank][head_dim]; wkv: [heads * head_dim][rank] */
  const float* mid_b;    /* rglru: [blocks * 2 * block_dim] interleaved; wkv: the decay's constant [heads * head_dim] */
  const uint16_t* uk_w;  /* latent: [heads * head_dim][rank] */
  const uint16_t* uv_w;  /* latent: [heads * v_dim][rank] */
  const uint16_t* o_w;   /* [D][mix_width] */
  const uint16_t* mlp_w; /* [2 ff][D], rows (gate_j, up_j) interleaved */
  const uint16_t* down_w;/* [D][ff] */
  const float* vec0;     /* rglru: -8 softplus(lam) [mix_width]; latent: weight of the latent's norm [rank];
                            wkv: weight behind the per-head norm [heads * head_dim] */
  const float* vec1;     /* rglru: convolution bias [mix_width]; wkv: bonus [heads * head_dim] */
  const float* vec2;     /* rglru: convolution taps [taps][mix_width]; wkv: mixes r, k, v, g, w [5][D] */
  const float* rope_cos; /* latent: [positions][rot_true / 2] */
  const float* rope_sin;
  const float* hc;       /* in1 [S], out1 [S], mix1 [S][S] ([from][to]), in2, out2, mix2 */
  const float* next1;    /* input weights of the sublayer that follows the mixer (ones behind the last one), [S] */
  const float* next2;    /* ... the feed-forward */
  void* cache;           /* latent: [slots][ring][rank + rot_dim], element type of the launch */
  float* state;          /* rglru: [slots][mix_width]; wkv: [slots][heads][head_dim (key)][head_dim (value)] */
  float* shift;          /* rglru: [slots][2][taps - 1][mix_width] last inputs of the convolution, oldest first;
                            wkv: [slots][2][D] the previous token's input.  The launch reads copy `flip`, writes 1 - flip */
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
  int32_t streams;
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
  int32_t reserved0;
  const uint16_t* embed;        /* bf16 [vocab_rows][D] */
  const float* final_norm;      /* [D] */
  const uint16_t* head;         /* bf16 [vocab_rows][D] */
  const int64_t* token_in;      /* prefill: [tokens]; decode: [1] */
  int64_t* token_out;           /* decode: the greedy token, or NULL */
  const int32_t* want;          /* prefill: [num_want] places in the portion */
  float* logits;                /* decode [vocab_rows]; prefill [num_want][vocab_rows] */
  float* layer_out;             /* prefill: [num_layers][tokens][D] sum of the streams behind each layer, or NULL */
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
