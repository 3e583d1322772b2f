// Internal interface between the kernels of the token language models and their step: lm.hip (context, parallel layers),
// sandwich.hip (sandwich layers), lm_gemm.hip (products), latent.hip and sigattn.hip (attention), scan.hip and gla.hip
// (recurrences), rows.hip (residual rows and norms), moe.hip (expert routing).
#pragma once
#include <vector>

#include "../../include/vui_lm.h"
#include "internal.h"

// Where the rows of a step live.  seq: rows are consecutive positions of one slot (host values); otherwise row m is
// the next position of slot slot_idx[m].
struct LmRows {
  const int32_t* slot_idx;
  const int32_t* seq_lens;
  int slot, pos0, seq;
  int S, n_slots;
};
#ifdef __HIPCC__
__device__ __forceinline__ int lm_slot(const LmRows& r, int m) {
  if (r.seq) return r.slot;
  const int s = r.slot_idx ? r.slot_idx[m] : m;
  return min(max(s, 0), r.n_slots - 1);
}
__device__ __forceinline__ int lm_pos(const LmRows& r, int m, int slot) { return r.seq ? r.pos0 + m : r.seq_lens[slot]; }
#endif

enum {
  LM_IN_ATTN = 0,   // everything an attention layer reads from h: queries, latent, key part, head gates, gated ff
  LM_IN_GRU_STEP,   // the same for a minGRU layer, one position per slot: the recurrence is the epilogue
  LM_IN_GRU_SEQ,    // ... positions of one sequence: update pairs for the scan
  LM_OUT,           // x += W y; operand copy and sums of squares of the new x
  LM_LOGITS,        // fp32 logits of chosen rows
  LM_EXPAND_K,      // keys of one head per blockIdx.z from cached latents
  LM_EXPAND_V,      // values, transposed
  // sandwich layers (rows arrive normed)
  LM_HEAD,          // LM_LOGITS without a row scale
  LM_PROJ,          // W x + bias in the context's dtype, row-major
  LM_PLAIN,         // the same in fp32
  LM_ACT,           // activation of an ungated feed-forward, tiled
  LM_MOE_UP,        // LM_ACT of the rows an expert was given, by tiles of the expert-sorted entries
  LM_MOE_DOWN,      // LM_PLAIN from those, one output row per (row, choice)
};

struct LmGemm {
  const void* X;  // (M x K) tiled
  const void* W;  // (N x K) tiled
  int M, N, K;    // N a multiple of 16, K of 64
  size_t wz;      // elements between the weights of consecutive blockIdx.z
  const int32_t* rowmap;  // row of X behind output row m, or nullptr
  int x_rows;             // rows of X (bound of rowmap)
  // row scale norm[0] / sqrt(sum(ssq[m]) / width + eps)
  const float* ssq;
  int np, width;
  float eps;
  const float* norm;
  LmRows rows;
  vui_lm_dims d;
  int mix_blocks;  // 16-row blocks of the mixer part of w_in; the gated feed-forward rows follow
  float limit;
  void* act;       // (M x out_k) tiled
  // attention: first block of each segment of w_in, rotated part, cache
  int b_qr, b_c, b_kr, b_g;
  int rot_pairs;
  const float* rope;
  void *qu, *qr;   // (heads, rows, dim64), (heads, rows, rot32)
  size_t qu_z, qr_z;
  float *craw, *gate;  // (rows, rank16), (rows, heads16)
  void* kr_cache;
  // minGRU
  const float *bz, *bx;
  float* state;
  float2* upd;     // (rows, gru16): {1 - z, z c}
  void* sg;        // (rows, gru16)
  // output
  float* x;        // (rows, w64) residual
  void* xt;        // (rows, w64) tiled
  float* ssq_out;
  float* layer_out;  // (rows, width) or nullptr
  // logits
  float* logits;
  int vocab;
  int32_t* upd_lens;
  const int32_t* upd_inc;
  int upd_rows;
  // expansion
  void* kv_out;
  size_t kv_z;
  // sandwich layers
  void* out;       // (rows, ldo) of the epilogue's type
  int ldo;
  const float* bias;  // (N) or nullptr
  int act_kind, act_k;  // VUI_LM_ACT_*, columns of act
  float act_pos, act_neg;
  // entries (row top + choice) sorted by expert, every expert's padded with -1 to whole tiles; expert of each tile
  const int32_t *ent, *tile_e, *n_tiles;
  int top, max_tiles, tile_rows;
  int sorted;      // X holds a row per entry instead of a row per position
};
int launch_lm_gemm(int dtype, int epi, const LmGemm& g, int nz, hipStream_t st);
int launch_lm_embed(int dtype, const int64_t* tokens, const void* table, float* x, void* xt, float* ssq, int rows, int width,
                    int w64, int np, int vocab, hipStream_t st);

// ---- latent attention (latent.hip) ----
struct LatentArgs {
  int dtype, M, heads;
  float scale;
  LmRows rows;
  vui_lm_dims d;
  int rank;
  // queries and latents of the new positions
  const void *qu, *qr;
  size_t qu_z, qr_z;
  void* qlat;      // (heads, rows, rank64)
  size_t qlat_z;
  const float* craw;
  const float* latent_norm;
  float eps;
  int own;         // the layer appends latents of its own
  const void *w_uk_t, *w_uv;
  void *c_cache, *kr_cache;
  // pieces (rows, heads, n_splits): unnormalised latent average (rank64), {max, sum}
  float *part, *part_ml;
  int n_splits;
  const float* gate;
  void* act;
  // expanded keys and values of one slot
  const void *kx, *vx;
  size_t kx_z, vx_z;
};
int launch_latent_append(const LatentArgs& a, hipStream_t st);   // norm + cache append of M rows
int launch_latent_query(const LatentArgs& a, hipStream_t st);    // queries into the latent space (+ append when own)
int launch_latent_attn(const LatentArgs& a, hipStream_t st);     // pieces
int launch_latent_value(const LatentArgs& a, hipStream_t st);    // merge, value expansion, head gate
int launch_latent_prefill_attn(const LatentArgs& a, hipStream_t st);  // expanded form, bf16
bool latent_mfma_ok(const vui_lm_dims& d);   // the matrix-core form of launch_latent_attn takes these sizes
bool latent_expand_ok(const vui_lm_dims& d);

// ---- gated recurrence over a sequence (scan.hip) ----
struct ScanArgs {
  int dtype, T, W, ld;      // channels W, row stride ld of upd / sg
  const float2* upd;        // {decay, input} per position and channel
  const void* gate;         // output gate
  float* state;             // (ld) of the slot
  int from_zero;
  float2* agg;              // (chunks + 1, ld)
  void* act;                // tiled output
  int out_k;
};
int launch_gated_scan(const ScanArgs& a, hipStream_t st);
#define LM_SCAN_CHUNK 32

// ---- expert routing: logits to choices, shares and entries sorted by expert ----
struct RouteArgs {
  int M, E, ldl, top, tile_rows;
  const float* logits;     // (M, ldl)
  int32_t* choice;         // (M, top)
  float* share;            // (M, top)
  int32_t *ent, *tile_e, *n_tiles;
};

// ---- residual rows of sandwich layers (rows.hip) ----
struct RowArgs {
  int dtype, M, width, w64, ldy, groups;
  float eps;
  // what the residual becomes, in this order of precedence
  const int64_t* tokens;   // embedding rows times emb_scale, copied to the second half of xcat too
  const void* embed;
  int vocab;
  float emb_scale;
  const float* step;       // y + step
  const float* post;       // x + norm(y) post; y the sum over `top` rows weighed by share, or one row (share nullptr)
  const float* y;
  const float* share;      // (M, top)
  int top;
  float* x;                // (rows, w64)
  float* layer_out;        // (M, width) or nullptr
  // what is left for the next product: the normed row, or the row itself in the first half of xcat
  const float* next;       // (w64) weight, or nullptr
  void* xt;                // (rows, w64) tiled
  void* xcat;              // (rows, 2 w64) tiled: [x | embedding]
  int to_cat;
  // router logits of the normed row (few rows), or rlog nullptr
  const void* w_router;
  const float* router_bias;
  int experts16;
  float* rlog;             // (M, experts16)
  RouteArgs route;         // of a single row: routed as well
};
int launch_lm_rows(const RowArgs& a, hipStream_t st);
bool lm_rows_routes(int M, int experts16);  // it takes the router's product too

// ---- attention with sigmoid weights (sigattn.hip) ----
struct SigAttnArgs {
  int dtype, M, heads, kv_heads, dim, vdim;
  float scale, eps;
  LmRows rows;
  vui_lm_dims d;
  const void* raw;         // (rows, ld): per head query, per group key and value, per head gate
  int ld;
  const float *q_norm, *k_norm;
  float temp_coef;
  int temp_every;
  const float* bias;       // (heads, bias_len)
  int bias_len;
  void *k_cache, *v_cache;
  void* q;                 // (heads, rows, dim64) tiled
  size_t q_z;
  float* part;             // (rows, heads, n_splits, vdim16)
  int n_splits;
  void* act;               // (rows, out_k) tiled
};
int launch_sig_prep(const SigAttnArgs& a, hipStream_t st);    // norms, temperature, append
int launch_sig_pieces(const SigAttnArgs& a, hipStream_t st);  // few rows: pieces, merge, gate
int launch_sig_prompt(const SigAttnArgs& a, hipStream_t st);  // block of one sequence, bf16
bool sig_mfma_ok(const vui_lm_dims& d);
bool sig_step_fused(int dtype, const LmRows& rows, const vui_lm_dims& d);  // launch_sig_pieces norms and appends by itself
int sig_splits(int M, int heads, int kv_heads);

// ---- gated linear attention (gla.hip) ----
struct GlaArgs {
  int dtype, M, heads, dim, vdim, rank;
  float eps, inv_tau, q_scale;
  LmRows rows;
  vui_lm_dims d;
  const void* raw;         // (rows, ld): per head query, key, value, gate; the low-rank part of the decay
  int ld;
  const float *w_a2, *a2_bias, *head_norm;
  float* state;            // (n_slots, heads, dim16, vdim16)
  float *bsum, *upd, *dec; // chunked form: (rows, heads, dim16), (chunks, heads, dim16, vdim16), (chunks, heads, dim16)
  void* act;
};
int launch_gla_step(const GlaArgs& a, hipStream_t st);   // one position per slot, or the positions of one sequence in turn
int launch_gla_chunk(const GlaArgs& a, hipStream_t st);  // positions of one sequence by chunks
bool gla_chunk_ok(const vui_lm_dims& d);
#define LM_GLA_CHUNK 32

// ---- expert routing (moe.hip) ----
int launch_moe_route(const RouteArgs& a, hipStream_t st);
// rows of a tiled operand (rows, cols) copied to their entries' places
int launch_moe_gather(int dtype, const RouteArgs& a, const void* x, void* out, int cols, int max_tiles, hipStream_t st);
// rows of the tiles an expert's entries are padded to
static inline int moe_tile_rows(int dtype, int M, int entries, int experts) {
  if (M <= 16) return 16;
  return dtype == VUI_DTYPE_BF16 && entries / experts >= 64 ? 64 : 32;
}
static inline int moe_max_tiles(int entries, int experts, int tile_rows) {
  const int a = entries / tile_rows + experts;
  return entries < a ? entries : a;
}

// ---- context ----
struct vui_lm_ctx {
  vui_lm_config c;
  vui_lm_weights w;
  std::vector<vui_lm_layer> layers;
  std::vector<vui_lm_dims> dims;
  int R16;  // rows of the activation buffers
  float* x; void* xt; float* ssq;
  void *qu, *qr, *qlat;
  float *craw, *gate, *part, *part_ml;
  void* act;
  float2* upd; void* sg; float2* agg;
  void *kx, *vx;
  float* layers_out;
  int expand_from;
  // sandwich layers
  void *xcat, *raw, *ffa, *xg;
  float *y, *bsum, *gupd, *gdec, *rlog, *share;
  int32_t *choice, *ent, *tile_e, *n_tiles;
  int attn_from, gla_from;
};
static inline int lm_pad(int v, int a) { return (v + a - 1) / a * a; }
static inline size_t lm_esz(const vui_lm_config& c) { return c.dtype == VUI_DTYPE_F32 ? 4 : 2; }
int sandwich_layer_dims(const vui_lm_config& c, const vui_lm_layer& L, vui_lm_dims* o);
int sandwich_check_layer(const vui_lm_config& c, const vui_lm_layer& L, int l);
bool sandwich_pointers_ok(const vui_lm_config& c, const vui_lm_layer& L);
size_t sandwich_carve(const vui_lm_config* c, const vui_lm_layer* layers, vui_lm_ctx* x, char* base);
int sandwich_layers(vui_lm_ctx* x, const int64_t* tokens, int M, const LmRows& rows, hipStream_t st);
