// Token language models: context, step and C ABI.  See include/vui_lm.h.
//
// Launches per layer: attention of few rows 5 (input projection; queries into the latent space + append; attention
// pieces; merge + value expansion; output projection), of a long block 6 (append, two expansions and one attention
// kernel in the middle); minGRU 2 for one position per slot, 3-4 for a sequence (the scan in the middle).
#include <string.h>

#include <new>

#include "lm.h"

#define LM_EXPAND_FROM 64  // positions of one call from which keys and values are expanded per head
#define LM_ATTN_FROM 64    // ... from which sigmoid attention takes blocks of a prompt
#define LM_GLA_FROM 5      // ... from which gated linear attention goes by chunks
#define LM_MAX_SPLITS 64   // latent_value_kernel keeps one piece per lane

#define pad lm_pad

static int lm_check_cfg(const vui_lm_config* c) {
  if (!c) { vui_set_error("config is NULL"); return VUI_EINVAL; }
  if (c->dtype != VUI_DTYPE_BF16 && c->dtype != VUI_DTYPE_F32) { vui_set_error("bad dtype %d", c->dtype); return VUI_EINVAL; }
  if (c->width < 1 || c->vocab < 1 || c->n_layers < 1 || c->n_layers > VUI_LM_MAX_LAYERS || c->max_seqlen < 1 || c->n_slots < 1 || c->max_rows < 1) {
    vui_set_error("lm: bad sizes width=%d vocab=%d layers=%d max_seqlen=%d slots=%d rows=%d", c->width, c->vocab, c->n_layers, c->max_seqlen, c->n_slots, c->max_rows);
    return VUI_EINVAL;
  }
  if (c->norm_groups < 0 || (c->norm_groups > 0 && c->width % c->norm_groups)) {
    vui_set_error("lm: a width of %d has no %d equal parts", c->width, c->norm_groups);
    return VUI_EINVAL;
  }
  return VUI_OK;
}

static bool lm_expands(const vui_lm_config& c, const vui_lm_dims& d) { return c.dtype == VUI_DTYPE_BF16 && latent_expand_ok(d); }

// n_splits of attention in the latent space: as many workgroups as stay resident beside each other (LDS holds two
// staged tiles of 32 latents per workgroup)
static int lm_splits(int M, int heads, int rank64) {
  const int t = (rank64 <= 256 ? 1024 : 512) / (M * ((heads + 15) / 16));
  return t < 1 ? 1 : (t > LM_MAX_SPLITS ? LM_MAX_SPLITS : t);
}

static size_t lm_carve(const vui_lm_config* c, const vui_lm_layer* layers, vui_lm_ctx* x, char* base) {
  if (c->norm_groups > 0) return sandwich_carve(c, layers, x, base);
  const size_t e = lm_esz(*c);
  const size_t R = pad(c->max_rows < 16 ? 16 : c->max_rows, 16);
  size_t qu = 0, qr = 0, ql = 0, cr = 0, ga = 0, pt = 0, pm = 0, ac = 0, up = 0, kx = 0, vx = 0;
  vui_lm_dims d;
  memset(&d, 0, sizeof(d));
  auto mx = [](size_t& a, size_t b) { if (b > a) a = b; };
  for (int l = 0; l < c->n_layers; ++l) {
    const vui_lm_layer& L = layers[l];
    vui_lm_layer_dims(c, &L, &d);
    mx(ac, R * d.out_k);
    if (L.mixer == VUI_LM_MINGRU) { mx(up, d.gru16); continue; }
    const size_t H = L.heads;
    mx(qu, H * R * d.dim64); mx(qr, H * R * d.rot32); mx(ql, H * R * d.rank64);
    mx(cr, R * d.rank16); mx(ga, R * d.heads16);
    size_t rows = R;  // rows x splits of attention pieces
    for (int M = 1; M <= (int)R && M <= 1024; ++M) mx(rows, (size_t)M * lm_splits(M, L.heads, d.rank64));
    mx(pt, rows * H * d.rank64); mx(pm, rows * H * 2);
    if (lm_expands(*c, d)) { mx(kx, H * d.s64 * d.dim64); mx(vx, H * d.s64 * d.vdim16); }
  }
  size_t off = 0;
  auto take = [&](size_t bytes) { size_t o = off; off += (bytes + 255) & ~(size_t)255; return o; };
#define TAKE(field, type, bytes) { const size_t o = take(bytes); if (x) x->field = (type)(base + o); }
  TAKE(x, float*, R * d.w64 * 4);
  TAKE(xt, void*, R * d.w64 * e);
  TAKE(ssq, float*, R * (d.w16 / 16) * 4);
  TAKE(qu, void*, qu * e);
  TAKE(qr, void*, qr * e);
  TAKE(qlat, void*, ql * e);
  TAKE(craw, float*, cr * 4);
  TAKE(gate, float*, ga * 4);
  TAKE(part, float*, pt * 4);
  TAKE(part_ml, float*, pm * 4);
  TAKE(act, void*, ac * e);
  TAKE(upd, float2*, R * up * 8);
  TAKE(sg, void*, R * up * e);
  TAKE(agg, float2*, (R / LM_SCAN_CHUNK + 2) * up * 8);
  TAKE(kx, void*, kx * e);
  TAKE(vx, void*, vx * e);
#undef TAKE
  return off;
}

static int lm_check_layer(const vui_lm_config& c, const vui_lm_layer& L, int l) {
  if (c.norm_groups > 0) return sandwich_check_layer(c, L, l);
  if (L.ff < 0) { vui_set_error("layer %d: ff %d", l, L.ff); return VUI_EINVAL; }
  if (L.mixer == VUI_LM_MINGRU) {
    if (L.rnn_width < 1) { vui_set_error("layer %d: recurrence width %d", l, L.rnn_width); return VUI_EINVAL; }
    return VUI_OK;
  }
  if (L.mixer != VUI_LM_LATENT_ATTENTION) { vui_set_error("layer %d: unknown mixer %d", l, L.mixer); return VUI_EINVAL; }
  if (L.heads < 1 || L.dim < 1 || L.rot_dim < 0 || L.rot_pairs < 0 || 2 * L.rot_pairs > L.rot_dim || L.vdim < 1 || L.kv_rank < 1 || L.kv_rank > 2048) {
    vui_set_error("layer %d: bad latent attention sizes heads=%d dim=%d rot=%d/%d vdim=%d rank=%d", l, L.heads, L.dim, L.rot_dim, L.rot_pairs, L.vdim, L.kv_rank);
    return VUI_EINVAL;
  }
  if (L.kv_from >= l) { vui_set_error("layer %d: kv_from %d does not come before it", l, L.kv_from); return VUI_EINVAL; }
  return VUI_OK;
}

extern "C" {

int vui_lm_layer_dims(const vui_lm_config* c, const vui_lm_layer* L, vui_lm_dims* o) {
  if (!c || !L || !o) { vui_set_error("NULL argument"); return VUI_EINVAL; }
  memset(o, 0, sizeof(*o));
  o->w16 = pad(c->width, 16); o->w64 = pad(c->width, 64); o->s64 = pad(c->max_seqlen, 64);
  if (c->norm_groups > 0) return sandwich_layer_dims(*c, *L, o);
  const bool attn = L->mixer == VUI_LM_LATENT_ATTENTION;
  const int tile = attn ? 32 : 48;  // rows of w_in a workgroup takes together
  int mix_k;
  if (attn) {
    o->dim16 = pad(L->dim, 16); o->dim64 = pad(L->dim, 64);
    o->rot16 = pad(L->rot_dim, 16); o->rot32 = pad(L->rot_dim < 1 ? 1 : L->rot_dim, 32);
    o->rank16 = pad(L->kv_rank, 16); o->rank64 = pad(L->kv_rank, 64);
    o->vdim16 = pad(L->vdim, 16); o->heads16 = pad(L->heads, 16);
    o->mix_rows = pad(L->heads * (o->dim16 + o->rot16) + (L->kv_from < 0 ? o->rank16 + o->rot16 : 0) + o->heads16, tile);
    mix_k = pad(L->heads * o->vdim16, 64);
  } else {
    o->gru16 = pad(L->rnn_width, 16);
    o->mix_rows = 3 * o->gru16;
    mix_k = pad(o->gru16, 64);
  }
  o->ff_pad = pad(L->ff, tile / 2);
  o->in_rows = o->mix_rows + 2 * o->ff_pad;
  o->ff_off = mix_k;
  o->out_k = mix_k + pad(o->ff_pad, 64);
  o->out_rows = o->w16;
  return VUI_OK;
}

int64_t vui_lm_workspace_bytes(const vui_lm_config* c, const vui_lm_layer* layers) {
  if (lm_check_cfg(c)) return VUI_EINVAL;
  if (!layers) { vui_set_error("NULL argument"); return VUI_EINVAL; }
  for (int l = 0; l < c->n_layers; ++l)
    if (lm_check_layer(*c, layers[l], l)) return VUI_EINVAL;
  return (int64_t)lm_carve(c, layers, nullptr, nullptr);
}

int vui_lm_create(const vui_lm_config* c, const vui_lm_layer* layers, const vui_lm_weights* w, void* workspace,
                  int64_t workspace_bytes, vui_lm_ctx** out) {
  if (!layers || !w || !workspace || !out) { vui_set_error("NULL argument"); return VUI_EINVAL; }
  const int64_t need = vui_lm_workspace_bytes(c, layers);
  if (need < 0) return VUI_EINVAL;
  if (workspace_bytes < need) { vui_set_error("workspace too small: %lld < %lld", (long long)workspace_bytes, (long long)need); return VUI_ENOMEM; }
  if (((uintptr_t)workspace) & 255) { vui_set_error("workspace must be 256-byte aligned"); return VUI_EINVAL; }
  if (!w->embed || !w->head || !w->final_norm) { vui_set_error("missing embedding, head or final norm"); return VUI_EINVAL; }
  for (int l = 0; l < c->n_layers; ++l) {
    const vui_lm_layer& L = layers[l];
    bool ok = L.w_in && L.w_out && (c->norm_groups > 0 || L.norm);
    if (c->norm_groups > 0) {
      ok = ok && sandwich_pointers_ok(*c, L);
    } else if (L.mixer == VUI_LM_MINGRU) {
      ok = ok && L.bias_z && L.bias_x && L.state;
    } else {
      ok = ok && L.w_uk_t && L.w_uv && L.c_cache && L.kr_cache && (L.rot_pairs == 0 || L.rope) && (L.kv_from >= 0 || L.latent_norm);
      vui_lm_dims d;
      vui_lm_layer_dims(c, &L, &d);
      if (lm_expands(*c, d)) ok = ok && L.w_uk;
      if (L.kv_from >= 0) {
        const vui_lm_layer& S = layers[L.kv_from];
        if (S.mixer != VUI_LM_LATENT_ATTENTION || S.kv_from >= 0 || S.kv_rank != L.kv_rank || S.rot_dim != L.rot_dim ||
            S.c_cache != L.c_cache || S.kr_cache != L.kr_cache) {
          vui_set_error("layer %d reads the latents of layer %d, which has none of its own or of another shape", l, L.kv_from);
          return VUI_EINVAL;
        }
      }
    }
    if (!ok) { vui_set_error("missing pointers of layer %d", l); return VUI_EINVAL; }
  }
  vui_lm_ctx* x = new (std::nothrow) vui_lm_ctx();
  if (!x) { vui_set_error("out of host memory"); return VUI_ENOMEM; }
  x->c = *c;
  x->w = *w;
  x->layers.assign(layers, layers + c->n_layers);
  x->dims.resize(c->n_layers);
  for (int l = 0; l < c->n_layers; ++l) vui_lm_layer_dims(c, &layers[l], &x->dims[l]);
  x->R16 = pad(c->max_rows < 16 ? 16 : c->max_rows, 16);
  x->layers_out = nullptr;
  x->expand_from = LM_EXPAND_FROM;
  x->attn_from = LM_ATTN_FROM;
  x->gla_from = LM_GLA_FROM;
  lm_carve(c, layers, x, (char*)workspace);
  *out = x;
  return VUI_OK;
}

void vui_lm_destroy(vui_lm_ctx* ctx) { delete ctx; }

int vui_lm_debug_layers(vui_lm_ctx* ctx, float* buf) {
  if (!ctx) { vui_set_error("NULL context"); return VUI_EINVAL; }
  ctx->layers_out = buf;
  return VUI_OK;
}

int vui_lm_expand_from(vui_lm_ctx* ctx, int rows) {
  if (!ctx) { vui_set_error("NULL context"); return VUI_EINVAL; }
  ctx->expand_from = rows > 0 ? rows : LM_EXPAND_FROM;
  return VUI_OK;
}

int vui_lm_block_from(vui_lm_ctx* ctx, int attn_rows, int gla_rows) {
  if (!ctx) { vui_set_error("NULL context"); return VUI_EINVAL; }
  ctx->attn_from = attn_rows > 0 ? attn_rows : LM_ATTN_FROM;
  ctx->gla_from = gla_rows > 0 ? gla_rows : LM_GLA_FROM;
  return VUI_OK;
}

}  // extern "C"

static int lm_attention(vui_lm_ctx* x, int l, int M, const LmRows& rows, LmGemm& g, hipStream_t st) {
  const vui_lm_layer& L = x->layers[l];
  const vui_lm_dims& d = x->dims[l];
  const vui_lm_config& c = x->c;
  const size_t e = lm_esz(c);
  const bool own = L.kv_from < 0;
  g.b_qr = L.heads * (d.dim16 / 16);
  g.b_c = g.b_qr + L.heads * (d.rot16 / 16);
  g.b_kr = g.b_c + (own ? d.rank16 / 16 : 0);
  g.b_g = g.b_kr + (own ? d.rot16 / 16 : 0);
  g.rot_pairs = L.rot_pairs; g.rope = L.rope;
  g.qu = x->qu; g.qr = x->qr; g.qu_z = (size_t)x->R16 * d.dim64; g.qr_z = (size_t)x->R16 * d.rot32;
  g.craw = x->craw; g.gate = x->gate; g.kr_cache = L.kr_cache;
  int rc = launch_lm_gemm(c.dtype, LM_IN_ATTN, g, 1, st);
  if (rc) return rc;

  LatentArgs a;
  memset(&a, 0, sizeof(a));
  a.dtype = c.dtype; a.M = M; a.heads = L.heads; a.scale = L.scale; a.rows = rows; a.d = d; a.rank = L.kv_rank;
  a.qu = x->qu; a.qr = x->qr; a.qu_z = g.qu_z; a.qr_z = g.qr_z;
  a.qlat = x->qlat; a.qlat_z = (size_t)x->R16 * d.rank64;
  a.craw = x->craw; a.latent_norm = L.latent_norm; a.eps = c.norm_eps; a.own = own;
  a.w_uk_t = L.w_uk_t; a.w_uv = L.w_uv; a.c_cache = L.c_cache; a.kr_cache = L.kr_cache;
  a.part = x->part; a.part_ml = x->part_ml; a.gate = x->gate; a.act = x->act;
  if (rows.seq && M >= x->expand_from && lm_expands(c, d)) {
    if (own && (rc = launch_latent_append(a, st))) return rc;
    LmGemm k;
    memset(&k, 0, sizeof(k));
    k.X = (const char*)L.c_cache + (size_t)rows.slot * d.s64 * d.rank64 * e;
    k.M = rows.pos0 + M; k.K = d.rank64; k.d = d; k.rows = rows;
    k.W = L.w_uk; k.N = d.dim64; k.wz = (size_t)d.dim64 * d.rank64; k.kv_out = x->kx; k.kv_z = (size_t)d.s64 * d.dim64;
    if ((rc = launch_lm_gemm(c.dtype, LM_EXPAND_K, k, L.heads, st))) return rc;
    k.W = L.w_uv; k.N = d.vdim16; k.wz = (size_t)d.vdim16 * d.rank64; k.kv_out = x->vx; k.kv_z = (size_t)d.s64 * d.vdim16;
    if ((rc = launch_lm_gemm(c.dtype, LM_EXPAND_V, k, L.heads, st))) return rc;
    a.kx = x->kx; a.vx = x->vx; a.kx_z = (size_t)d.s64 * d.dim64; a.vx_z = (size_t)d.s64 * d.vdim16;
    return launch_latent_prefill_attn(a, st);
  }
  a.n_splits = lm_splits(M, L.heads, d.rank64);
  if ((rc = launch_latent_query(a, st))) return rc;
  if ((rc = launch_latent_attn(a, st))) return rc;
  return launch_latent_value(a, st);
}

static int lm_recurrence(vui_lm_ctx* x, int l, int M, const LmRows& rows, LmGemm& g, hipStream_t st) {
  const vui_lm_layer& L = x->layers[l];
  const vui_lm_dims& d = x->dims[l];
  g.bz = L.bias_z; g.bx = L.bias_x; g.state = L.state; g.upd = x->upd; g.sg = x->sg;
  int rc = launch_lm_gemm(x->c.dtype, rows.seq ? LM_IN_GRU_SEQ : LM_IN_GRU_STEP, g, 1, st);
  if (rc || !rows.seq) return rc;
  ScanArgs s;
  memset(&s, 0, sizeof(s));
  s.dtype = x->c.dtype; s.T = M; s.W = d.gru16; s.ld = d.gru16; s.upd = x->upd; s.gate = x->sg;
  s.state = L.state + (size_t)rows.slot * d.gru16; s.from_zero = rows.pos0 == 0; s.agg = x->agg; s.act = x->act; s.out_k = d.out_k;
  return launch_gated_scan(s, st);
}

static int lm_layers(vui_lm_ctx* x, const int64_t* tokens, int M, const LmRows& rows, hipStream_t st) {
  const vui_lm_config& c = x->c;
  if (c.norm_groups > 0) return sandwich_layers(x, tokens, M, rows, st);
  const int w64 = x->dims[0].w64, np = x->dims[0].w16 / 16;
  int rc = launch_lm_embed(c.dtype, tokens, x->w.embed, x->x, x->xt, x->ssq, M, c.width, w64, np, c.vocab, st);
  if (rc) return rc;
  for (int l = 0; l < c.n_layers; ++l) {
    const vui_lm_layer& L = x->layers[l];
    const vui_lm_dims& d = x->dims[l];
    LmGemm g;
    memset(&g, 0, sizeof(g));
    g.X = x->xt; g.W = L.w_in; g.M = M; g.N = d.in_rows; g.K = d.w64; g.x_rows = M;
    g.ssq = x->ssq; g.np = np; g.width = c.width; g.eps = c.norm_eps; g.norm = L.norm;
    g.rows = rows; g.d = d; g.mix_blocks = d.mix_rows / 16; g.limit = L.limit; g.act = x->act;
    rc = L.mixer == VUI_LM_MINGRU ? lm_recurrence(x, l, M, rows, g, st) : lm_attention(x, l, M, rows, g, st);
    if (rc) return rc;
    LmGemm o;
    memset(&o, 0, sizeof(o));
    o.X = x->act; o.W = L.w_out; o.M = M; o.N = d.out_rows; o.K = d.out_k; o.d = d; o.rows = rows;
    o.x = x->x; o.xt = x->xt; o.ssq_out = x->ssq; o.np = np; o.width = c.width;
    o.layer_out = x->layers_out ? x->layers_out + (size_t)l * M * c.width : nullptr;
    if ((rc = launch_lm_gemm(c.dtype, LM_OUT, o, 1, st))) return rc;
  }
  return VUI_OK;
}

static LmGemm lm_logits(vui_lm_ctx* x, const LmRows& rows, int M, int x_rows, const int32_t* rowmap, float* out) {
  LmGemm g;
  memset(&g, 0, sizeof(g));
  const vui_lm_dims& d = x->dims[0];
  g.X = x->xt; g.W = x->w.head; g.M = M; g.N = pad(x->c.vocab, 16); g.K = d.w64; g.rowmap = rowmap; g.x_rows = x_rows;
  g.ssq = x->ssq; g.np = d.w16 / 16; g.width = x->c.width; g.eps = x->c.norm_eps; g.norm = x->w.final_norm;
  g.rows = rows; g.d = d; g.logits = out; g.vocab = x->c.vocab;
  return g;
}

__global__ void lm_set_len_kernel(int32_t* seq_lens, int slot, int v) { seq_lens[slot] = v; }

extern "C" {

int vui_lm_decode(vui_lm_ctx* x, const int64_t* tokens, const int32_t* slot_idx, int32_t* seq_lens, const int32_t* seq_inc,
                  int B, float* logits_out, vui_stream_t stream) {
  if (!x) { vui_set_error("NULL context"); return VUI_EINVAL; }
  if (!tokens || !seq_lens || !logits_out) { vui_set_error("vui_lm_decode: NULL argument"); return VUI_EINVAL; }
  if (B < 1 || B > VUI_MAX_BATCH || (!slot_idx && B > x->c.n_slots)) { vui_set_error("vui_lm_decode: B=%d", B); return VUI_EINVAL; }
  hipStream_t st = (hipStream_t)stream;
  LmRows r;
  memset(&r, 0, sizeof(r));
  r.slot_idx = slot_idx; r.seq_lens = seq_lens; r.S = x->c.max_seqlen; r.n_slots = x->c.n_slots;
  int rc = lm_layers(x, tokens, B, r, st);
  if (rc) return rc;
  LmGemm g = lm_logits(x, r, B, B, nullptr, logits_out);
  g.upd_lens = seq_lens; g.upd_inc = seq_inc; g.upd_rows = B;
  return launch_lm_gemm(x->c.dtype, x->c.norm_groups > 0 ? LM_HEAD : LM_LOGITS, g, 1, st);
}

int vui_lm_prefill(vui_lm_ctx* x, const int64_t* tokens, int T, int slot, int pos0, int32_t* seq_lens, const int32_t* want,
                   int n_want, float* logits_out, vui_stream_t stream) {
  if (!x) { vui_set_error("NULL context"); return VUI_EINVAL; }
  if (!tokens || !seq_lens || n_want < 0 || (n_want > 0 && (!want || !logits_out))) { vui_set_error("vui_lm_prefill: bad argument"); return VUI_EINVAL; }
  if (T < 1 || T > x->c.max_rows) { vui_set_error("vui_lm_prefill: %d positions outside [1, %d]", T, x->c.max_rows); return VUI_EINVAL; }
  if (slot < 0 || slot >= x->c.n_slots) { vui_set_error("vui_lm_prefill: slot %d outside [0, %d)", slot, x->c.n_slots); return VUI_EINVAL; }
  if (pos0 < 0 || pos0 + T > x->c.max_seqlen) { vui_set_error("vui_lm_prefill: positions %d..%d outside the slot (%d)", pos0, pos0 + T, x->c.max_seqlen); return VUI_EINVAL; }
  hipStream_t st = (hipStream_t)stream;
  LmRows r;
  memset(&r, 0, sizeof(r));
  r.seq = 1; r.slot = slot; r.pos0 = pos0; r.S = x->c.max_seqlen; r.n_slots = x->c.n_slots;
  int rc = lm_layers(x, tokens, T, r, st);
  if (rc) return rc;
  if (n_want > 0 && (rc = launch_lm_gemm(x->c.dtype, x->c.norm_groups > 0 ? LM_HEAD : LM_LOGITS, lm_logits(x, r, n_want, T, want, logits_out), 1, st))) return rc;
  hipLaunchKernelGGL(lm_set_len_kernel, dim3(1), dim3(1), 0, st, seq_lens, slot, pos0 + T);
  HIP_TRY(hipGetLastError());
  return VUI_OK;
}

int vui_sample_tokens(const float* logits, int vocab, float* rep_counts, int32_t* rep_hist, int32_t* rep_pos, float penalty,
                      int window, const vui_sample_params* sp, int64_t* out, int B, vui_stream_t stream) {
  if (!logits || !sp || !out || B < 1) { vui_set_error("vui_sample_tokens: bad argument"); return VUI_EINVAL; }
  if (window > 0 && rep_counts && penalty > 1.0f && (!rep_hist || !rep_pos)) { vui_set_error("a repetition window needs rep_hist and rep_pos"); return VUI_EINVAL; }
  SampleArgs s;
  memset(&s, 0, sizeof(s));
  s.dtype = VUI_DTYPE_F32; s.logits = logits; s.rep_counts = rep_counts; s.rep_hist = rep_hist; s.rep_pos = rep_pos;
  s.penalty = penalty; s.window = window; s.temperature = sp->temperature; s.top_k = sp->top_k; s.top_p = sp->top_p;
  s.seed = sp->seed; s.frame_ctr = sp->frame_ctr; s.state_rows = sp->state_rows; s.dev = sp->dev;
  s.exact_k = sp->keep_ties ? 0 : 1; s.CS = vocab; s.B = B; s.out = out; s.out_stride = 1;
  return vocab > 8192 ? launch_sample_wide(s, (hipStream_t)stream) : launch_sample(s, (hipStream_t)stream);  // what sample_kernel holds in registers
}

}  // extern "C"
