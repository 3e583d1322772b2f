/*
 * vui_lm.h - C ABI of the token language models: decoder-only models whose layers are described one by one (which
 * mixer, which sizes, which feed-forward) and run on the same library, slots and sampler as the Vui backbone.
 * No counterpart in the reference.
 *
 * Two forms of layers (vui_lm_config.norm_groups):
 *   parallel (0): x <- x + mixer(h) + ff(h) with h = norm(x), an RMS norm with a scalar weight;
 *   sandwich (n >= 1): x <- x + norm(mixer(norm(x))), then x <- x + norm(ff(norm(x))), every norm over n equal
 *     consecutive parts of the vector with one weight per entry.
 * A model that runs some of its layers several times lists every run as a layer of its own: the same weights, but
 * caches and states of its own.
 *
 * The residual stream, norms, positions and angles, attention scores and weights, routers, gates of a recurrence and
 * its state are fp32; products, cached latents, keys and values are of the context's dtype with fp32 accumulation.
 *
 * Conventions as in vui_amd.h: caller-owned device memory, work enqueued on the given stream without waiting,
 * 0 or a negative VUI_E* code, vui_last_error().  vui_lm_decode may be recorded into a HIP graph.
 *
 * Matrices arrive in the tiled operand layout (blocks of 16 rows x 64 columns in lane order, vui_amd/csrc/tile.h;
 * vui_amd/lm_layout.py writes it), padded with zero rows and columns to the sizes vui_lm_layer_dims gives.
 */
#ifndef VUI_LM_H
#define VUI_LM_H

#include "vui_amd.h"

#ifdef __cplusplus
extern "C" {
#endif

#define VUI_LM_MAX_LAYERS 1024
/* mixers; the first two belong to parallel layers, the others to sandwich layers */
#define VUI_LM_LATENT_ATTENTION 0
#define VUI_LM_MINGRU 1
#define VUI_LM_GLA 2
#define VUI_LM_SIGMOID_ATTENTION 3
/* activations of an ungated feed-forward */
#define VUI_LM_ACT_XIELU 0   /* z > 0: act_pos z^2 + z / 2, else act_neg (exp(z) - 1 - z) + z / 2 */
#define VUI_LM_ACT_RELU2 1
#define VUI_LM_MAX_TOP 16    /* experts a token uses */
#define VUI_LM_MAX_EXPERTS 1024

typedef struct vui_lm_config {
  int32_t dtype;      /* VUI_DTYPE_*: weights, activations and caches */
  int32_t width, vocab, n_layers;
  int32_t max_seqlen; /* positions of a slot */
  int32_t n_slots;
  int32_t max_rows;   /* most positions of one vui_lm_prefill call (sizes the workspace) */
  float norm_eps;
  int32_t norm_groups; /* 0: parallel layers; else sandwich layers with norms over this many parts */
  float embed_scale;   /* sandwich layers: the embedding is multiplied by this */
} vui_lm_config;

typedef struct vui_lm_layer {
  int32_t mixer;      /* VUI_LM_* */
  /* latent attention: the cache holds per position the normed latent (kv_rank) and one rotated key part (rot_dim)
   * common to the heads; heads expand keys (dim) and values (vdim) from the latent */
  int32_t kv_from;    /* layer whose latents are read, or -1: the layer has a down-projection of its own */
  int32_t heads, dim, rot_dim, rot_pairs, vdim, kv_rank;
  float scale;
  /* minGRU: S_t = (1 - z) S_(t-1) + z c, z and c from the current token only */
  int32_t rnn_width;
  /* feed-forward g sigmoid(1.702 g) (u + 1), g clamped from above and u on both sides; ff = 0: none */
  int32_t ff;
  float limit;
  const float* norm;      /* (1) weight of the layer's norm */
  const void* w_in;       /* (in_rows, w64) tiled: everything that reads h; row order in vui_amd/lm_layout.py */
  const void* w_out;      /* (out_rows, out_k) tiled: mixer and feed-forward output side by side along k */
  const void* w_uk_t;     /* (heads, rank16, dim64) tiled: per head, latent <- unrotated query */
  const void* w_uk;       /* (heads, dim64, rank64) tiled: per head, key <- latent (bf16 contexts) */
  const void* w_uv;       /* (heads, vdim16, rank64) tiled: per head, value <- latent */
  const float* latent_norm; /* (rank16) */
  const float* rope;      /* (max_seqlen, rot_pairs, 2) cos/sin */
  const float *bias_z, *bias_x; /* (gru16) */
  void* c_cache;          /* (n_slots, s64, rank64) tiled rows: latents; of layer kv_from when that is set */
  void* kr_cache;         /* (n_slots, s64, rot32) tiled rows (32-column blocks): rotated key parts */
  float* state;           /* (n_slots, gru16) fp32; gated linear attention (n_slots, heads, dim16, vdim16) */

  /* ---- sandwich layers ----
   * sigmoid attention (heads, kv_heads, dim, vdim, scale): queries and keys normed per head, the query times
   * 1 + temp_coef ln(floor((p + 1) / temp_every) + 1) at position p, weights sigmoid(score scale + bias), where the
   * bias is a table over the distance that stays at its last entry beyond it.
   * gated linear attention (heads, dim, vdim, rank): S <- diag(a) S + k v^T, a = sigmoid(W_a2 W_a1 h + b)^inv_tau */
  int32_t kv_heads, temp_every, bias_len, rank;
  float temp_coef, inv_tau;
  /* ungated feed-forward of ff features per expert; experts = 0: one dense feed-forward */
  int32_t act, experts, top;
  float act_pos, act_neg;
  const float *norm1, *norm1b, *norm2, *norm2b; /* (w64), zero beyond width */
  const float *in_bias, *out_bias;              /* (in_rows), (out_rows), or NULL */
  const float *q_norm, *k_norm;                 /* (dim16) */
  const float* dist_bias;                       /* (heads, bias_len): distances 0 .. bias_len - 1 and beyond */
  void *k_cache;                                /* (n_slots, kv_heads, s64, dim64) tiled rows */
  void *v_cache;                                /* (n_slots, kv_heads, s64 / 32, vdim16 / 16) blocks of 16 dims x 32 positions */
  const float *w_a2, *a2_bias;                  /* (heads, dim16, rank), (heads, dim16) */
  const float* head_norm;                       /* (vdim16) */
  const void *w_up, *w_down;                    /* (experts or 1, ff16, w64), (experts or 1, out_rows, ff64) tiled */
  const void* w_router;                         /* (experts16, w64) tiled */
  const float* router_bias;                     /* (experts16) */
  const void* loop_in;                          /* (out_rows, 2 w64) tiled or NULL: x <- loop_in [x; embedding] + loop_step ahead of the layer */
  const float* loop_step;                       /* (w64) */
} vui_lm_layer;

/* Padded sizes of a layer's operands (all derived from the configuration). */
typedef struct vui_lm_dims {
  int32_t w16, w64, s64;
  int32_t dim16, dim64, rot16, rot32, rank16, rank64, vdim16, heads16;
  int32_t gru16;
  int32_t mix_rows, in_rows; /* rows of w_in: mixer part, all */
  int32_t ff_pad, ff_off;    /* feed-forward columns (padded) and where they start inside out_k */
  int32_t out_k, out_rows;
  int32_t ff16, ff64, experts16;
} vui_lm_dims;

typedef struct vui_lm_weights {
  const void* embed;       /* (vocab, width) row-major */
  const void* head;        /* (vocab padded to 32, w64) tiled */
  const float* final_norm; /* (1); sandwich layers (w64) */
} vui_lm_weights;

typedef struct vui_lm_ctx vui_lm_ctx;

int vui_lm_layer_dims(const vui_lm_config* cfg, const vui_lm_layer* layer, vui_lm_dims* out);
/* Zero-filled device memory a context needs (activations of max_rows positions, attention pieces, expanded keys). */
int64_t vui_lm_workspace_bytes(const vui_lm_config* cfg, const vui_lm_layer* layers);
int vui_lm_create(const vui_lm_config* cfg, const vui_lm_layer* layers, const vui_lm_weights* w, void* workspace,
                  int64_t workspace_bytes, vui_lm_ctx** out);
void vui_lm_destroy(vui_lm_ctx* ctx);

/* One token for each of B rows (B <= VUI_MAX_BATCH).  tokens device (B) int64; slot_idx device (B) int32 or NULL (the
 * identity); seq_lens device (n_slots) int32: position of each slot's token, advanced afterwards by seq_inc
 * (n_slots) or, where that is NULL, by one for the B rows' slots.  A recurrence starts from zero at position 0,
 * whatever its state holds.  logits_out device (B, vocab) fp32. */
int vui_lm_decode(vui_lm_ctx* ctx, const int64_t* tokens, const int32_t* slot_idx, int32_t* seq_lens,
                  const int32_t* seq_inc, int B, float* logits_out, vui_stream_t stream);

/* T tokens (T <= max_rows) of one slot at positions pos0 .. pos0 + T - 1; seq_lens[slot] becomes pos0 + T.
 * want device (n_want) int32: which of the T positions' logits are written to logits_out (n_want, vocab) fp32. */
int vui_lm_prefill(vui_lm_ctx* ctx, const int64_t* tokens, int T, int slot, int pos0, int32_t* seq_lens,
                   const int32_t* want, int n_want, float* logits_out, vui_stream_t stream);

/* Test aid: the residual stream behind each layer, for the calls that follow, goes to buf (n_layers, rows of the call,
 * width) fp32; NULL switches it off. */
int vui_lm_debug_layers(vui_lm_ctx* ctx, float* buf);
/* Test and measurement aid: positions of one call from which attention expands keys and values per head instead of
 * attending in the latent space (0 restores the default). */
int vui_lm_expand_from(vui_lm_ctx* ctx, int rows);
/* The same for sandwich layers: positions of one call from which attention takes blocks of a prompt, and a gated linear
 * attention its chunked form (0 restores the defaults). */
int vui_lm_block_from(vui_lm_ctx* ctx, int attn_rows, int gla_rows);

/* vui_sample_cb0 without a context: one token per row from fp32 logits (B, vocab), vocab up to 524288. */
int vui_sample_tokens(const float* logits, int vocab, float* rep_counts, int32_t* rep_hist, int32_t* rep_pos,
                      float penalty, int window, const vui_sample_params* sp, int64_t* out, int B, vui_stream_t stream);

#ifdef __cplusplus
}
#endif
#endif /* VUI_LM_H */
