/* C ABI of libmoshi_tlm.so: token language models on MI355X (gfx950).  Same conventions as moshi_mi.h - device pointers unless said
 * otherwise, work enqueued on the caller's stream, status codes with mmi_last_error(), a handle bound to the device current at create. */
#ifndef MOSHI_TLM_H_
#define MOSHI_TLM_H_
#include "moshi_mi.h"
#ifdef __cplusplus
extern "C" {
#endif

/* ------------------------------------------------------------------------------------------ */
/* Token language models: decoder-only networks over token ids (libmoshi_tlm.so)              */
/* ------------------------------------------------------------------------------------------ */
/* The layers are data: each has one mixer and one feed-forward reading norms of the same input (parallel sublayers), optional layer
 * scales, grouped RMS norms, an optional run of layers repeated with the same weights.  Sequences live in slots; their attention cache
 * is a pool of pages of mmi_tlm_info(MMI_TLM_PAGE_TOKENS) tokens, their recurrent state one entry per slot and recurrent layer run. */

/* mixers */
#define MMI_TLM_MIX_LATENT_ATTENTION 1
#define MMI_TLM_MIX_MINGRU 2
#define MMI_TLM_MIX_ATTENTION 3         /* softmax attention, query heads share key/value heads */
#define MMI_TLM_MIX_CHANNEL_DELTA 4     /* gated delta rule, one decay per key channel */
#define MMI_TLM_MIX_LIGHTNING 5         /* linear attention, one constant decay per head */
/* feed-forwards */
#define MMI_TLM_MLP_NONE 0
#define MMI_TLM_MLP_MOE 1
#define MMI_TLM_MLP_DENSE 2             /* gated: gate and up projections, down projection */
/* feed-forward activations */
#define MMI_TLM_ACT_RELU2 1
#define MMI_TLM_ACT_CLAMPED_SWIGLU 2    /* g = min(gate, limit), u = clamp(up, +-limit): g sigmoid(1.702 g) (u + 1) */
/* routers */
#define MMI_TLM_ROUTE_TOKEN_TABLE 1
/* what the passes of the repeated layers start with */
#define MMI_TLM_LOOP_ADD 0              /* the second and later ones: x + embedding */
#define MMI_TLM_LOOP_PROJECT 1          /* every one: loop.in [x; embedding] + loop.step[pass] */

typedef struct mmi_tlm_layer {
    int32_t mixer;
    int32_t width;                                /* minGRU: channels */
    int32_t heads, dim, vdim, rot_dim;            /* latent attention: per head un-rotated / value / rotated dimensions */
    int32_t q_rank, kv_rank;
    int32_t window;                               /* keys seen, the position itself included; 0 = all earlier ones */
    float scale;
    double rot_base;
    int32_t mlp, experts, top, ff, act, router;
    int32_t kv_heads;                             /* attention, channel delta: key/value (query/key) heads */
    int32_t keep_first;                           /* attention with a window: first positions that stay visible */
    int32_t sink;                                 /* attention: one is added to the softmax denominator */
    int32_t conv;                                 /* channel delta: taps of the short convolutions */
    int32_t decay_rank, gate_rank;                /* channel delta: ranks of the decay's and the gate's projection */
    const double* decay;                          /* lightning: [heads], host */
    float limit;                                  /* clamped SwiGLU */
} mmi_tlm_layer;

typedef struct mmi_tlm_cfg {
    int32_t vocab, width, n_layers;
    const mmi_tlm_layer* layers;
    int32_t loop_start, loop_stop, loop_times;    /* layers [start, stop) run `times` times; start == stop: no repetition */
    int32_t norm_groups;
    float norm_eps, logit_scale;
    int32_t loop_inject, norms, layer_scales;     /* norms 2: the feed-forward has a norm of its own; layer_scales: ls1 / ls2 exist */
    int32_t tied_head;                            /* logits from the (unscaled) embedding table */
    float embed_scale;
    int32_t bigram_buckets;                       /* 0: no bigram embedding; row (previous mul_prev + token mul_cur) mod buckets, first token: row `buckets` */
    int64_t bigram_mul_prev, bigram_mul_cur;
    int32_t max_positions;                        /* 0: no learned positions; otherwise also the longest sequence */
    int32_t dtype;                                /* MMI_BF16 or MMI_F32: operands of the matrix products, activations and cache */
} mmi_tlm_cfg;

typedef struct mmi_tlm mmi_tlm;

/* Tensors are bf16 (tables int32), device pointers, copied or repacked: `embed`, `bigram`, `pos`, `head`, `final.norm`, `loop.in`,
 * `loop.step`, per layer `l<i>.norm1`, `.norm2`, `.ls1`, `.ls2`, `.mix.*`, `.mlp.*`.  max_slots: live sequences; max_tokens: cache pool (rounded up to pages); max_step_tokens: tokens of
 * one step. */
int mmi_tlm_create(const mmi_tlm_cfg* cfg, const mmi_tensor_desc* weights, int32_t n_weights, int32_t max_slots, int64_t max_tokens,
                   int32_t max_step_tokens, mmi_tlm** out);
void mmi_tlm_destroy(mmi_tlm* m);
/* Admit a sequence (MMI_ERR_BUSY when every slot is taken) / give back what it holds. */
int mmi_tlm_open(mmi_tlm* m, int32_t* slot);
int mmi_tlm_close(mmi_tlm* m, int32_t slot);
/* One batch: entry e appends counts[e] tokens to slot slots[e] (each slot at most once).  tokens: host, concatenated; -1 = the token
 * mmi_tlm_sample last drew for that slot.  want: host, ascending rows of the concatenation whose logits are written to `logits`
 * (device fp32 [n_want][vocab]).  MMI_ERR_BUSY, with nothing changed, when the pool has too few free pages. */
int mmi_tlm_step(mmi_tlm* m, int32_t n_entries, const int32_t* slots, const int32_t* counts, const int32_t* tokens, int32_t n_want,
                 const int32_t* want, float* logits, mmi_stream stream);
/* Draw one token per row of device fp32 logits [n][vocab]; row i belongs to slot slots[i] and uses temp[i] / top_k[i] (temp <= 0:
 * greedy).  out: device int32 [n]. */
int mmi_tlm_sample(mmi_tlm* m, int32_t n, const float* logits, const int32_t* slots, const float* temp, const int32_t* top_k, uint64_t seed,
                   int32_t* out, mmi_stream stream);
/* Bookkeeping: pool and slots.  MMI_TLM_POSITION / MMI_TLM_HELD_PAGES take a slot. */
#define MMI_TLM_PAGE_TOKENS 0
#define MMI_TLM_TOTAL_PAGES 1
#define MMI_TLM_FREE_PAGES 2
#define MMI_TLM_FREE_SLOTS 3
#define MMI_TLM_POSITION 4
#define MMI_TLM_HELD_PAGES 5
#define MMI_TLM_WEIGHT_BYTES 6
#define MMI_TLM_LAYER_RUNS 7
#define MMI_TLM_GRAPHS 8
int64_t mmi_tlm_info(const mmi_tlm* m, int32_t which, int32_t slot);
/* Pages a sequence would have to be given to grow from its position by n tokens (slot < 0: from an empty slot). */
int64_t mmi_tlm_pages_needed(const mmi_tlm* m, int32_t slot, int64_t n);
/* Residual stream after every layer run of the next steps: taps = device fp32 [layer runs][tokens of the step][width], or NULL. */
int mmi_tlm_set_taps(mmi_tlm* m, float* taps);
/* "site\tkernel\tbytes" per launch of the last step. */
int64_t mmi_tlm_launch_list(const mmi_tlm* m, char* buf, int64_t cap);

#ifdef __cplusplus
}
#endif
#endif /* MOSHI_TLM_H_ */
