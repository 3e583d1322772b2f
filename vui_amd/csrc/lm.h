// Internal interface between the kernels of the token language models (lm_gemm.hip, latent.hip, scan.hip) and their
// step (lm.hip).
#pragma once
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
