// Sandwich layers of the token language models: x <- x + norm(mixer(norm(x))), then x <- x + norm(ff(norm(x))).  See
// include/vui_lm.h and lm.hip, which holds the context and the C ABI.
//
// Launches: input projection, mixer (sigmoid attention 2, portions of a prompt 3, blocks of one 2; gated linear
// attention 1, by chunks 3), output projection, rows, up, down, rows; an expert layer adds 1 for routing (none for one row), with more
// rows than 16 the router's product, 2 for routing and 1 that puts the rows in order.
// The rows launch (rows.hip) norms and adds what a sublayer produced and norms what the next one reads.
#include <string.h>

#include "lm.h"

static int mix_rows_of(const vui_lm_layer& L, const vui_lm_dims& d) {
  if (L.mixer == VUI_LM_GLA) return L.heads * 2 * (d.dim16 + d.vdim16) + lm_pad(L.rank, 16);
  return L.heads * d.dim16 + L.kv_heads * (d.dim16 + d.vdim16) + d.heads16;
}

int sandwich_layer_dims(const vui_lm_config& c, const vui_lm_layer& L, vui_lm_dims* o) {
  o->dim16 = lm_pad(L.dim, 16); o->dim64 = lm_pad(L.dim, 64);
  o->vdim16 = lm_pad(L.vdim, 16); o->heads16 = lm_pad(L.heads, 16);
  o->mix_rows = o->in_rows = lm_pad(mix_rows_of(L, *o), 32);
  o->out_k = lm_pad(L.heads * o->vdim16, 64);
  o->out_rows = o->w16;
  o->ff16 = lm_pad(L.ff, 16); o->ff64 = lm_pad(L.ff, 64);
  o->experts16 = lm_pad(L.experts, 16);
  return VUI_OK;
}

int sandwich_check_layer(const vui_lm_config& c, const vui_lm_layer& L, int l) {
  if (L.mixer != VUI_LM_GLA && L.mixer != VUI_LM_SIGMOID_ATTENTION) { vui_set_error("layer %d: mixer %d does not go with sandwich layers", l, L.mixer); return VUI_EINVAL; }
  if (L.heads < 1 || L.dim < 1 || L.vdim < 1 || L.dim > 2048 || L.vdim > 2048) {
    vui_set_error("layer %d: bad sizes heads=%d dim=%d vdim=%d", l, L.heads, L.dim, L.vdim);
    return VUI_EINVAL;
  }
  if (L.mixer == VUI_LM_GLA ? L.rank < 1 : (L.kv_heads < 1 || L.heads % L.kv_heads || L.bias_len < 1 || (L.temp_coef != 0.f && L.temp_every < 1))) {
    vui_set_error("layer %d: bad mixer constants kv_heads=%d bias_len=%d temp_every=%d rank=%d", l, L.kv_heads, L.bias_len, L.temp_every, L.rank);
    return VUI_EINVAL;
  }
  if (L.ff < 0 || L.experts < 0 || L.experts > VUI_LM_MAX_EXPERTS || (L.experts > 0 && (L.ff < 1 || L.top < 1 || L.top > L.experts || L.top > VUI_LM_MAX_TOP))) {
    vui_set_error("layer %d: bad feed-forward ff=%d experts=%d top=%d", l, L.ff, L.experts, L.top);
    return VUI_EINVAL;
  }
  return VUI_OK;
}

bool sandwich_pointers_ok(const vui_lm_config& c, const vui_lm_layer& L) {
  bool ok = L.norm1 && L.norm1b && (!L.loop_in == !L.loop_step);
  if (L.mixer == VUI_LM_GLA) ok = ok && L.w_a2 && L.a2_bias && L.head_norm && L.state;
  else ok = ok && L.q_norm && L.k_norm && L.dist_bias && L.k_cache && L.v_cache;
  if (L.ff > 0) ok = ok && L.norm2 && L.norm2b && L.w_up && L.w_down;
  if (L.experts > 0) ok = ok && L.w_router && L.router_bias;
  return ok;
}

size_t sandwich_carve(const vui_lm_config* c, const vui_lm_layer* layers, vui_lm_ctx* x, char* base) {
  const size_t e = lm_esz(*c);
  const size_t R = lm_pad(c->max_rows < 16 ? 16 : c->max_rows, 16);
  size_t q = 0, raw = 0, ac = 0, pt = 0, ff = 0, yr = R, bs = 0, up = 0, de = 0, rl = 0, ch = 0, en = 0, ti = 0, xg = 0;
  bool loops = false;
  vui_lm_dims d;
  memset(&d, 0, sizeof(d));
  auto mx = [](size_t& a, size_t b) { if (b > a) a = b; };
  for (int l = 0; l < c->n_layers; ++l) {
    const vui_lm_layer& L = layers[l];
    vui_lm_layer_dims(c, &L, &d);
    const size_t H = L.heads;
    loops = loops || L.loop_in;
    mx(ac, R * d.out_k); mx(raw, R * d.in_rows);
    if (L.mixer == VUI_LM_GLA) {
      const size_t nc = (R + LM_GLA_CHUNK - 1) / LM_GLA_CHUNK;
      if (gla_chunk_ok(d)) { mx(bs, R * H * d.dim16); mx(up, nc * H * d.dim16 * d.vdim16); mx(de, nc * H * d.dim16); }
    } else {
      mx(q, H * R * d.dim64);
      size_t rows = R;  // rows x splits of attention pieces
      for (int M = 1; M <= (int)R && M <= 1024; ++M) mx(rows, (size_t)M * sig_splits(M, L.heads, L.kv_heads));
      mx(pt, rows * H * d.vdim16);
    }
    if (L.experts > 0) {
      const size_t n = R * L.top;
      for (int tr = 16; tr <= 64; tr *= 2) {
        const size_t tiles = moe_max_tiles(n, L.experts, tr), rows = tiles * tr;
        mx(ff, rows * d.ff64); mx(en, rows); mx(ti, tiles);
        if (tr > 16) mx(xg, rows * d.w64);
      }
      mx(yr, n); mx(ch, n); mx(rl, R * d.experts16);
    } else {
      mx(ff, R * d.ff64);
    }
  }
  size_t off = 0;
  auto take = [&](size_t bytes) { size_t o = off; off += (bytes + 255) & ~(size_t)255; return o; };
#define TAKE(field, type, bytes) { const size_t o = take(bytes); if (x) x->field = (type)(base + o); }
  TAKE(x, float*, R * d.w64 * 4);
  TAKE(xt, void*, R * d.w64 * e);
  TAKE(xcat, void*, loops ? R * 2 * d.w64 * e : 0);
  TAKE(raw, void*, raw * e);
  TAKE(qu, void*, q * e);
  TAKE(part, float*, pt * 4);
  TAKE(act, void*, ac * e);
  TAKE(y, float*, yr * d.w16 * 4);
  TAKE(ffa, void*, ff * e);
  TAKE(xg, void*, xg * e);
  TAKE(bsum, float*, bs * 4);
  TAKE(gupd, float*, up * 4);
  TAKE(gdec, float*, de * 4);
  TAKE(rlog, float*, rl * 4);
  TAKE(share, float*, ch * 4);
  TAKE(choice, int32_t*, ch * 4);
  TAKE(ent, int32_t*, en * 4);
  TAKE(tile_e, int32_t*, ti * 4);
  TAKE(n_tiles, int32_t*, 4);
#undef TAKE
  return off;
}

// C = X W^T of M rows
static LmGemm product(const vui_lm_ctx* x, const vui_lm_dims& d, const LmRows& rows, const void* X, const void* W, int M, int N, int K) {
  LmGemm g;
  memset(&g, 0, sizeof(g));
  g.X = X; g.W = W; g.M = M; g.N = N; g.K = K; g.x_rows = M; g.d = d; g.rows = rows; g.width = x->c.width;
  return g;
}

static int plain(const vui_lm_ctx* x, const vui_lm_dims& d, const LmRows& rows, const void* X, const void* W, const float* bias, int M, int N, int K, float* y, hipStream_t st) {
  LmGemm g = product(x, d, rows, X, W, M, N, K);
  g.bias = bias; g.out = y; g.ldo = N;
  return launch_lm_gemm(x->c.dtype, LM_PLAIN, g, 1, st);
}

static int mixer(vui_lm_ctx* x, int l, int M, const LmRows& rows, hipStream_t st) {
  const vui_lm_layer& L = x->layers[l];
  const vui_lm_dims& d = x->dims[l];
  LmGemm g = product(x, d, rows, x->xt, L.w_in, M, d.in_rows, d.w64);
  g.bias = L.in_bias; g.out = x->raw; g.ldo = d.in_rows;
  int rc = launch_lm_gemm(x->c.dtype, LM_PROJ, g, 1, st);
  if (rc) return rc;
  if (L.mixer == VUI_LM_GLA) {
    GlaArgs a;
    memset(&a, 0, sizeof(a));
    a.dtype = x->c.dtype; a.M = M; a.heads = L.heads; a.dim = L.dim; a.vdim = L.vdim; a.rank = L.rank;
    a.eps = x->c.norm_eps; a.inv_tau = L.inv_tau; a.q_scale = L.scale; a.rows = rows; a.d = d;
    a.raw = x->raw; a.ld = d.in_rows; a.w_a2 = L.w_a2; a.a2_bias = L.a2_bias; a.head_norm = L.head_norm;
    a.state = L.state; a.bsum = x->bsum; a.upd = x->gupd; a.dec = x->gdec; a.act = x->act;
    rc = rows.seq && M >= x->gla_from && gla_chunk_ok(d) && L.rank <= 512 ? launch_gla_chunk(a, st) : launch_gla_step(a, st);
  } else {
    SigAttnArgs a;
    memset(&a, 0, sizeof(a));
    a.dtype = x->c.dtype; a.M = M; a.heads = L.heads; a.kv_heads = L.kv_heads; a.dim = L.dim; a.vdim = L.vdim;
    a.scale = L.scale; a.eps = x->c.norm_eps; a.rows = rows; a.d = d; a.raw = x->raw; a.ld = d.in_rows;
    a.q_norm = L.q_norm; a.k_norm = L.k_norm; a.temp_coef = L.temp_coef; a.temp_every = L.temp_every < 1 ? 1 : L.temp_every;
    a.bias = L.dist_bias; a.bias_len = L.bias_len; a.k_cache = L.k_cache; a.v_cache = L.v_cache;
    a.q = x->qu; a.q_z = (size_t)x->R16 * d.dim64; a.part = x->part; a.act = x->act;
    if (!sig_step_fused(x->c.dtype, rows, d) && (rc = launch_sig_prep(a, st))) return rc;
    if (rows.seq && M >= x->attn_from && x->c.dtype == VUI_DTYPE_BF16 && sig_mfma_ok(d)) {
      rc = launch_sig_prompt(a, st);
    } else {
      a.n_splits = sig_splits(M, L.heads, L.kv_heads);
      rc = launch_sig_pieces(a, st);
    }
  }
  if (rc) return rc;
  return plain(x, d, rows, x->act, L.w_out, L.out_bias, M, d.out_rows, d.out_k, x->y, st);
}

static RouteArgs routing(const vui_lm_ctx* x, int l, int M) {
  const vui_lm_layer& L = x->layers[l];
  RouteArgs r;
  memset(&r, 0, sizeof(r));
  r.M = M; r.E = L.experts; r.ldl = x->dims[l].experts16; r.top = L.top; r.tile_rows = moe_tile_rows(x->c.dtype, M, M * L.top, L.experts);
  r.logits = x->rlog; r.choice = x->choice; r.share = x->share; r.ent = x->ent; r.tile_e = x->tile_e; r.n_tiles = x->n_tiles;
  return r;
}

// leaves the outputs in y: one row per position, or per (position, choice) of an expert layer
static int feed_forward(vui_lm_ctx* x, int l, int M, const LmRows& rows, hipStream_t st) {
  const vui_lm_layer& L = x->layers[l];
  const vui_lm_dims& d = x->dims[l];
  int rc;
  LmGemm up = product(x, d, rows, x->xt, L.w_up, M, d.ff16, d.w64);
  up.act = x->ffa; up.act_k = d.ff64; up.act_kind = L.act; up.act_pos = L.act_pos; up.act_neg = L.act_neg;
  if (L.experts == 0) {
    if ((rc = launch_lm_gemm(x->c.dtype, LM_ACT, up, 1, st))) return rc;
    return plain(x, d, rows, x->ffa, L.w_down, nullptr, M, d.out_rows, d.ff64, x->y, st);
  }
  if (!lm_rows_routes(M, d.experts16) && (rc = plain(x, d, rows, x->xt, L.w_router, L.router_bias, M, d.experts16, d.w64, x->rlog, st))) return rc;
  const RouteArgs r = routing(x, l, M);
  if (!lm_rows_routes(M, d.experts16) || M > 1) {
    if ((rc = launch_moe_route(r, st))) return rc;
  }
  up.ent = x->ent; up.tile_e = x->tile_e; up.n_tiles = x->n_tiles; up.top = L.top; up.wz = (size_t)d.ff16 * d.w64;
  up.tile_rows = r.tile_rows;
  up.max_tiles = moe_max_tiles(M * L.top, L.experts, r.tile_rows);
  if (M > 16) {
    if ((rc = launch_moe_gather(x->c.dtype, r, x->xt, x->xg, d.w64, up.max_tiles, st))) return rc;
    up.X = x->xg; up.sorted = 1;
  }
  if ((rc = launch_lm_gemm(x->c.dtype, LM_MOE_UP, up, 1, st))) return rc;
  LmGemm down = product(x, d, rows, x->ffa, L.w_down, M, d.out_rows, d.ff64);
  down.ent = x->ent; down.tile_e = x->tile_e; down.n_tiles = x->n_tiles; down.top = L.top; down.wz = (size_t)d.out_rows * d.ff64;
  down.max_tiles = up.max_tiles; down.tile_rows = r.tile_rows; down.out = x->y; down.ldo = d.out_rows;
  return launch_lm_gemm(x->c.dtype, LM_MOE_DOWN, down, 1, st);
}

int sandwich_layers(vui_lm_ctx* x, const int64_t* tokens, int M, const LmRows& rows, hipStream_t st) {
  const vui_lm_config& c = x->c;
  const int n = c.n_layers;
  RowArgs r;
  memset(&r, 0, sizeof(r));
  r.dtype = c.dtype; r.M = M; r.width = c.width; r.w64 = x->dims[0].w64; r.ldy = x->dims[0].w16; r.groups = c.norm_groups;
  r.eps = c.norm_eps; r.x = x->x; r.xt = x->xt; r.y = x->y; r.vocab = c.vocab; r.embed = x->w.embed; r.emb_scale = c.embed_scale;
  bool loops = false;
  for (int l = 0; l < n; ++l) loops = loops || x->layers[l].loop_in;
  r.xcat = loops ? x->xcat : nullptr;
  // what the row launch ahead of layer l leaves: the operand of the loop's mixing product, or the normed row
  auto ahead = [&](int l) {
    r.to_cat = l < n && x->layers[l].loop_in;
    r.next = r.to_cat ? nullptr : (l < n ? x->layers[l].norm1 : x->w.final_norm);
  };
  ahead(0);
  RowArgs emb = r;
  emb.tokens = tokens;
  int rc = launch_lm_rows(emb, st);
  for (int l = 0; l < n && !rc; ++l) {
    const vui_lm_layer& L = x->layers[l];
    const vui_lm_dims& d = x->dims[l];
    if (L.loop_in) {
      if ((rc = plain(x, d, rows, x->xcat, L.loop_in, nullptr, M, d.out_rows, 2 * d.w64, x->y, st))) return rc;
      RowArgs s = r;
      s.step = L.loop_step; s.next = L.norm1; s.to_cat = 0; s.layer_out = nullptr;
      if ((rc = launch_lm_rows(s, st))) return rc;
    }
    if ((rc = mixer(x, l, M, rows, st))) return rc;
    float* lo = x->layers_out ? x->layers_out + (size_t)l * M * c.width : nullptr;
    r.share = nullptr; r.post = L.norm1b; r.layer_out = nullptr;
    if (L.ff > 0) {
      r.next = L.norm2; r.to_cat = 0;
      RowArgs mid = r;
      if (L.experts > 0 && lm_rows_routes(M, d.experts16)) {
        mid.w_router = L.w_router; mid.router_bias = L.router_bias; mid.experts16 = d.experts16; mid.rlog = x->rlog;
        mid.route = routing(x, l, M);
      }
      if ((rc = launch_lm_rows(mid, st))) return rc;
      if ((rc = feed_forward(x, l, M, rows, st))) return rc;
      r.post = L.norm2b;
      if (L.experts > 0) { r.share = x->share; r.top = L.top; }
    }
    r.layer_out = lo;
    ahead(l + 1);
    if ((rc = launch_lm_rows(r, st))) return rc;
  }
  return rc;
}
