// Attention whose weights are sigmoids of the scores: nothing is normalised over the keys, so pieces of a key range
// simply add up.  Queries and keys are normed per head, a query is scaled by a temperature that grows with its
// position, and a score gets a bias from a table over the distance.
//
// A decode step norms and appends inside the kernel of the pieces; portions of a prompt do it in a launch of their own.
//
// Caches: keys as tiled rows (tile.h), so that 16 keys x 64 columns are an operand of the matrix cores as they lie;
// values in blocks of 16 dims x 32 positions, an operand of the second product.
#include "common.h"
#include "lm.h"
#include "tile.h"

// element of the value cache of one slot and group
__device__ __forceinline__ size_t val_off(int pos, int d, int nvb) {
  return ((size_t)(pos >> 5) * nvb + (d >> 4)) * 512 + ((d & 15) + 16 * ((pos & 15) >> 2)) * 8 + 4 * ((pos & 31) >> 4) + (pos & 3);
}

// columns of a projected row
struct SigCols { int k, v, g; };
__device__ __forceinline__ SigCols sig_cols(const SigAttnArgs& p) {
  SigCols c;
  c.k = p.heads * p.d.dim16;
  c.v = c.k + p.kv_heads * p.d.dim16;
  c.g = c.v + p.kv_heads * p.d.vdim16;
  return c;
}

__device__ __forceinline__ float sig_temp(const SigAttnArgs& p, int pos) {
  return p.temp_coef == 0.f ? 1.f : 1.0f + p.temp_coef * logf((float)((pos + 1) / p.temp_every + 1));
}

// ---- norms, temperature, append; one wave per (row, query head | key group | value group) ----
template <typename T>
__global__ __launch_bounds__(256) void sig_prep_kernel(const SigAttnArgs p) {
  const int lane = threadIdx.x & 63, m = blockIdx.y;
  const int u = blockIdx.x * 4 + __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
  const SigCols c = sig_cols(p);
  const int slot = lm_slot(p.rows, m), pos = lm_pos(p.rows, m, slot);
  if (u >= p.heads + 2 * p.kv_heads || pos < 0 || pos >= p.rows.S) return;
  const T* row = (const T*)p.raw + (size_t)m * p.ld;
  if (u >= p.heads + p.kv_heads) {
    const int g = u - p.heads - p.kv_heads, nvb = p.d.vdim16 >> 4;
    T* dst = (T*)p.v_cache + ((size_t)slot * p.kv_heads + g) * p.d.s64 * p.d.vdim16;
    for (int k = lane; k < p.d.vdim16; k += 64) dst[val_off(pos, k, nvb)] = row[c.v + g * p.d.vdim16 + k];
    return;
  }
  const bool q = u < p.heads;
  const T* src = row + (q ? u * p.d.dim16 : c.k + (u - p.heads) * p.d.dim16);
  float ss = 0.f;
  for (int k = lane * 4; k < p.d.dim16; k += 256) {  // columns beyond dim hold zeros
#pragma unroll
    for (int i = 0; i < 4; ++i) { const float v = El<T>::ld(src + k + i); ss = fmaf(v, v, ss); }
  }
  ss = wave_sum(ss);
  const float r = (q ? sig_temp(p, pos) : 1.f) / sqrtf(ss / (float)p.dim + p.eps);
  const float* w = q ? p.q_norm : p.k_norm;
  T* dst = q ? (T*)p.q + u * p.q_z : (T*)p.k_cache + ((size_t)slot * p.kv_heads + (u - p.heads)) * p.d.s64 * p.d.dim64;
  const int at = q ? m : pos;
  for (int k = lane * 4; k < p.d.dim64; k += 256) {
    float o[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) o[i] = k < p.d.dim16 ? El<T>::ld(src + k + i) * r * w[k + i] : 0.f;
    Tl<T>::st4(dst + tl_off<T>(at, k, p.d.dim64), o);
  }
}

// A row that sees len keys is cut into pieces of this many (whole 32-key tiles), at most ns of them.
#define SIG_PIECE 128
__device__ __forceinline__ int sig_chunk(int len, int ns) { return max(((len + ns - 1) / ns + 31) & ~31, SIG_PIECE); }

// ---- pieces, any sizes: one workgroup per (row, head, piece); fp32 arithmetic ----
#define SIG_TILE 256
template <typename T>
__global__ __launch_bounds__(256) void sig_piece_kernel(const SigAttnArgs p) {
  extern __shared__ __align__(16) float lq[];  // query (dim64), accumulators (vdim16)
  __shared__ float sc[SIG_TILE];
  const int m = blockIdx.x, h = blockIdx.y, sp = blockIdx.z, tid = threadIdx.x;
  const int g = h / (p.heads / p.kv_heads), nvb = p.d.vdim16 >> 4, D = p.d.dim64;
  const int slot = lm_slot(p.rows, m), pos = lm_pos(p.rows, m, slot);
  const int len = min(max(pos + 1, 1), p.rows.S);
  const int chunk = sig_chunk(len, p.n_splits), lo = min(sp * chunk, len), hi = min(lo + chunk, len);
  if (lo >= hi) return;  // no such piece: the merge does not look for it
  float* acc = lq + D;
  for (int k = tid; k < D; k += 256) lq[k] = El<T>::ld((const T*)p.q + h * p.q_z + tl_off<T>(m, k, D));
  for (int k = tid; k < p.d.vdim16; k += 256) acc[k] = 0.f;
  const T* kc = (const T*)p.k_cache + ((size_t)slot * p.kv_heads + g) * p.d.s64 * D;
  const T* vc = (const T*)p.v_cache + ((size_t)slot * p.kv_heads + g) * p.d.s64 * p.d.vdim16;
  const float* bias = p.bias + (size_t)h * p.bias_len;
  __syncthreads();
  for (int j0 = lo; j0 < hi; j0 += SIG_TILE) {
    const int j = j0 + tid, nj = min(SIG_TILE, hi - j0);
    float w = 0.f;
    if (j < hi) {
      float s = 0.f;
      constexpr int EP = Tl<T>::EP;
      for (int k = 0; k < D; k += EP) {
        const T* q = kc + tl_off<T>(j, k, D);
#pragma unroll
        for (int e = 0; e < EP; ++e) s = fmaf(lq[k + e], El<T>::ld(q + e), s);
      }
      w = 1.0f / (1.0f + expf(-(s * p.scale + bias[min(len - 1 - j, p.bias_len - 1)])));
    }
    sc[tid] = w;
    __syncthreads();
    for (int d = tid; d < p.d.vdim16; d += 256) {
      float a = acc[d];
      for (int k = 0; k < nj; ++k) a = fmaf(sc[k], El<T>::ld(vc + val_off(j0 + k, d, nvb)), a);
      acc[d] = a;
    }
    __syncthreads();
  }
  float* out = p.part + (((size_t)m * p.heads + h) * p.n_splits + sp) * p.d.vdim16;
  for (int d = tid; d < p.d.vdim16; d += 256) out[d] = acc[d];
}

// ---- one tile of 32 keys on the matrix cores (bf16): DB = dim64 / 64, VT >= vdim16 / 16 ----
// Scores^T (keys x 16 columns) leave a lane with eight keys of one column, which is operand layout for
// out^T = V^T w^T; the fp32 weights go in as a bf16 pair (value and remainder).
template <int DB, int VT>
struct SigTile {
  uint4 kf[2][2 * DB], vf[VT];
  __device__ __forceinline__ void load(const bf16_t* kb, const bf16_t* vb, int k0, int nvb) {
#pragma unroll
    for (int t = 0; t < 2; ++t)
#pragma unroll
      for (int i = 0; i < 2 * DB; ++i) kf[t][i] = *reinterpret_cast<const uint4*>(kb + (size_t)((k0 >> 4) + t) * DB * 1024 + i * 512);
#pragma unroll
    for (int d = 0; d < VT; ++d) vf[d] = *reinterpret_cast<const uint4*>(vb + ((size_t)(k0 >> 5) * nvb + min(d, nvb - 1)) * 512);
  }
  __device__ __forceinline__ void scores(const uint4* qf, tl_f32x4* sc) const {
#pragma unroll
    for (int t = 0; t < 2; ++t) {
      sc[t] = tl_f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int i = 0; i < 2 * DB; ++i) sc[t] = Tl<bf16_t>::mma(kf[t][i], qf[i], sc[t]);
    }
  }
  __device__ __forceinline__ void add(const float* w, tl_f32x4* acc) const {
    uint4 hi, lo;
    hi.x = f2bf2(w[0], w[1]); hi.y = f2bf2(w[2], w[3]); hi.z = f2bf2(w[4], w[5]); hi.w = f2bf2(w[6], w[7]);
    lo.x = f2bf2(w[0] - bf_lo(hi.x), w[1] - bf_hi(hi.x)); lo.y = f2bf2(w[2] - bf_lo(hi.y), w[3] - bf_hi(hi.y));
    lo.z = f2bf2(w[4] - bf_lo(hi.z), w[5] - bf_hi(hi.z)); lo.w = f2bf2(w[6] - bf_lo(hi.w), w[7] - bf_hi(hi.w));
#pragma unroll
    for (int d = 0; d < VT; ++d) {
      acc[d] = Tl<bf16_t>::mma(vf[d], hi, acc[d]);
      acc[d] = Tl<bf16_t>::mma(vf[d], lo, acc[d]);
    }
  }
};

#define SIG_LOG2E 1.4426950408889634f
// sigmoid of a score given t = -log2(e) score
__device__ __forceinline__ float sig_weight(float t) { return __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(t)); }

// a normed row as a lane's part of an operand: columns 64 b + 16 kg .. + 15 in f[2 b], f[2 b + 1]; src: dim16 values
template <int DB>
__device__ __forceinline__ void sig_normed(const bf16_t* src, const float* w, int dim16, int dim, float eps, float mul, int kg, uint4* f) {
  float v[DB][16], ss = 0.f;
#pragma unroll
  for (int b = 0; b < DB; ++b) {
    const int col = b * 64 + kg * 16;
    const bool live = col < dim16;
    const uint4* q = reinterpret_cast<const uint4*>(src + (live ? col : 0));
    const uint4 x[2] = {q[0], q[1]};
#pragma unroll
    for (int h = 0; h < 2; ++h) {
      const uint32_t u[4] = {x[h].x, x[h].y, x[h].z, x[h].w};
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        v[b][8 * h + 2 * i] = live ? bf_lo(u[i]) : 0.f;
        v[b][8 * h + 2 * i + 1] = live ? bf_hi(u[i]) : 0.f;
      }
    }
#pragma unroll
    for (int i = 0; i < 16; ++i) ss = fmaf(v[b][i], v[b][i], ss);
  }
  const float r = mul / sqrtf(rows_sum(ss) / (float)dim + eps);
#pragma unroll
  for (int b = 0; b < DB; ++b) {
    const int col = b * 64 + kg * 16;
    const float* c = w + (col < dim16 ? col : 0);
#pragma unroll
    for (int i = 0; i < 16; ++i) v[b][i] *= r * c[i];
#pragma unroll
    for (int h = 0; h < 2; ++h)
      f[2 * b + h] = make_uint4(f2bf2(v[b][8 * h], v[b][8 * h + 1]), f2bf2(v[b][8 * h + 2], v[b][8 * h + 3]),
                                f2bf2(v[b][8 * h + 4], v[b][8 * h + 5]), f2bf2(v[b][8 * h + 6], v[b][8 * h + 7]));
  }
}

// ---- pieces on the matrix cores (bf16): one workgroup per (row, up to 16 heads of one group, piece) ----
// STEP (one position per slot): queries are normed here, and the wave that comes to the new position's tile norms its key,
// puts key and value into its operands and appends them (workgroups of further heads of the group write the same).
template <int DB, int VT, bool STEP>
__global__ __launch_bounds__(256) void sig_piece_mfma_kernel(const SigAttnArgs p) {
  __shared__ __align__(16) float s_acc[4][VT * 256];
  const int tid = threadIdx.x, wave = __builtin_amdgcn_readfirstlane(tid >> 6), lane = tid & 63, l16 = lane & 15, kg = lane >> 4;
  const int m = blockIdx.x, sp = blockIdx.z, per = p.heads / p.kv_heads, nhb = (per + 15) >> 4;
  const int g = (int)blockIdx.y / nhb, h0 = g * per + ((int)blockIdx.y % nhb) * 16, nh = min(16, (g + 1) * per - h0);
  const int head = h0 + min(l16, nh - 1), nvb = p.d.vdim16 >> 4;
  const int slot = lm_slot(p.rows, m), pos = lm_pos(p.rows, m, slot);
  const int len = min(max(pos + 1, 1), p.rows.S);
  const int chunk = sig_chunk(len, p.n_splits), lo = min(sp * chunk, len), hi = min(lo + chunk, len);
  if (lo >= hi) return;  // no such piece
  const bf16_t* kb = (const bf16_t*)p.k_cache + ((size_t)slot * p.kv_heads + g) * p.d.s64 * (DB * 64) + lane * 8;
  const bf16_t* vb = (const bf16_t*)p.v_cache + ((size_t)slot * p.kv_heads + g) * p.d.s64 * p.d.vdim16 + lane * 8;
  const float* bias = p.bias + (size_t)head * p.bias_len;
  uint4 qf[2 * DB];
  const bf16_t* row = (const bf16_t*)p.raw + (size_t)m * p.ld;
  if (STEP) {
    sig_normed<DB>(row + head * p.d.dim16, p.q_norm, p.d.dim16, p.dim, p.eps, sig_temp(p, pos), kg, qf);
  } else {
#pragma unroll
    for (int i = 0; i < 2 * DB; ++i)
      qf[i] = *reinterpret_cast<const uint4*>((const bf16_t*)p.q + head * p.q_z + ((size_t)(m >> 4) * DB * 2 + i) * 512 + ((m & 15) + 16 * kg) * 8);
  }
  tl_f32x4 acc[VT];
#pragma unroll
  for (int d = 0; d < VT; ++d) acc[d] = tl_f32x4{0.f, 0.f, 0.f, 0.f};
  const float c = -p.scale * SIG_LOG2E;
  for (int k0 = lo + 32 * wave; k0 < hi; k0 += 128) {
    SigTile<DB, VT> t;
    t.load(kb, vb, k0, nvb);
    float b[8], w[8];
#pragma unroll
    for (int e = 0; e < 8; ++e) {
      const int j = k0 + 16 * (e >> 2) + 4 * kg + (e & 3);
      b[e] = bias[min(max(len - 1 - j, 0), p.bias_len - 1)];
    }
    if (STEP && pos == len - 1 && (pos >> 5) == (k0 >> 5)) {  // uniform; a position outside the slot is not stored
      const SigCols cols = sig_cols(p);
      uint4 nk[2 * DB];
      sig_normed<DB>(row + cols.k + g * p.d.dim16, p.k_norm, p.d.dim16, p.dim, p.eps, 1.f, kg, nk);
      const bool mine = l16 == (pos & 15);
      bf16_t* ko = const_cast<bf16_t*>(kb) + (size_t)(pos >> 4) * DB * 1024;
#pragma unroll
      for (int i = 0; i < 2 * DB; ++i) {
        if (mine && !(pos & 16)) t.kf[0][i] = nk[i];
        if (mine && (pos & 16)) t.kf[1][i] = nk[i];
        if (mine) *reinterpret_cast<uint4*>(ko + i * 512) = nk[i];
      }
      const bool vmine = kg == ((pos & 15) >> 2);
      const int w = 2 * ((pos & 31) >> 4) + ((pos & 3) >> 1), sh = 16 * (pos & 1), e = 4 * ((pos & 31) >> 4) + (pos & 3);
      bf16_t* vo = const_cast<bf16_t*>(vb) + (size_t)(pos >> 5) * nvb * 512 + e;
#pragma unroll
      for (int d = 0; d < VT; ++d) {
        const bf16_t nv = row[cols.v + g * p.d.vdim16 + min(d, nvb - 1) * 16 + l16];
        const uint32_t keep = 0xffffu << (16 - sh), put = (uint32_t)nv << sh;
        if (vmine && w == 0) t.vf[d].x = (t.vf[d].x & keep) | put;
        if (vmine && w == 1) t.vf[d].y = (t.vf[d].y & keep) | put;
        if (vmine && w == 2) t.vf[d].z = (t.vf[d].z & keep) | put;
        if (vmine && w == 3) t.vf[d].w = (t.vf[d].w & keep) | put;
        if (vmine && d < nvb) vo[(size_t)d * 512] = nv;
      }
    }
    __builtin_amdgcn_sched_barrier(0);
    tl_f32x4 s[2];
    t.scores(qf, s);
#pragma unroll
    for (int e = 0; e < 8; ++e) {
      const int j = k0 + 16 * (e >> 2) + 4 * kg + (e & 3);
      w[e] = j < hi ? sig_weight(fmaf(s[e >> 2][e & 3], c, -SIG_LOG2E * b[e])) : 0.f;
    }
    t.add(w, acc);
  }
#pragma unroll
  for (int d = 0; d < VT; ++d) *reinterpret_cast<tl_f32x4*>(&s_acc[wave][(d * 64 + lane) * 4]) = acc[d];
  __syncthreads();
  for (int sl = tid; sl < nvb * 64; sl += 256) {
    const int d = sl >> 6, hh = sl & 15, k4 = (sl >> 4) & 3;
    if (hh >= nh) continue;
    tl_f32x4 o = *reinterpret_cast<const tl_f32x4*>(&s_acc[0][sl * 4]);
#pragma unroll
    for (int w = 1; w < 4; ++w) o += *reinterpret_cast<const tl_f32x4*>(&s_acc[w][sl * 4]);
    *reinterpret_cast<tl_f32x4*>(p.part + (((size_t)m * p.heads + h0 + hh) * p.n_splits + sp) * p.d.vdim16 + 16 * d + 4 * k4) = o;
  }
}

// ---- sum of the pieces and head gate; a thread owns four value columns of a row ----
template <typename T>
__global__ __launch_bounds__(256) void sig_merge_kernel(const SigAttnArgs p) {
  const int m = blockIdx.y, col = (blockIdx.x * 256 + threadIdx.x) * 4;
  if (col >= p.heads * p.d.vdim16) return;
  const int h = col / p.d.vdim16, d = col - h * p.d.vdim16;
  const float gate = El<T>::ld((const T*)p.raw + (size_t)m * p.ld + sig_cols(p).g + h);
  const int slot = lm_slot(p.rows, m), pos = lm_pos(p.rows, m, slot);
  const int len = min(max(pos + 1, 1), p.rows.S);
  const int chunk = sig_chunk(len, p.n_splits), np = (len + chunk - 1) / chunk;  // pieces that exist
  const float* pc = p.part + ((size_t)m * p.heads + h) * p.n_splits * p.d.vdim16 + d;
  tl_f32x4 o = {0.f, 0.f, 0.f, 0.f};
  for (int s0 = 0; s0 < np; s0 += 8) {
    tl_f32x4 v[8];
#pragma unroll
    for (int u = 0; u < 8; ++u) v[u] = *reinterpret_cast<const tl_f32x4*>(pc + (size_t)min(s0 + u, np - 1) * p.d.vdim16);
#pragma unroll
    for (int u = 0; u < 8; ++u)
      if (s0 + u < np) o += v[u];
  }
  const float f = 1.0f / (1.0f + expf(-gate));
  const float r[4] = {o[0] * f, o[1] * f, o[2] * f, o[3] * f};
  Tl<T>::st4((T*)p.act + tl_off<T>(m, col, p.d.out_k), r);
}

// ---- block of one sequence (bf16): one workgroup per 32 queries and head, waves take 32 keys in turn ----
#define SIGP_WAVES (VT <= 4 ? 8 : 4)
#define SIG_BIAS_LDS 4096  // longest table that is copied to LDS
template <int DB, int VT>
__global__ __launch_bounds__(64 * SIGP_WAVES) void sig_prompt_kernel(const SigAttnArgs p) {
  extern __shared__ __align__(16) float lb[];  // table times -log2(e), when it fits
  __shared__ __align__(16) float s_acc[SIGP_WAVES][VT * 256];
  const int tid = threadIdx.x, wave = __builtin_amdgcn_readfirstlane(tid >> 6), lane = tid & 63, l16 = lane & 15, kg = lane >> 4;
  const int qt = gridDim.x - 1 - blockIdx.x, h = blockIdx.y;  // the tiles with the most keys start first
  const int g = h / (p.heads / p.kv_heads), q0 = qt * 32, nvb = p.d.vdim16 >> 4, pos0 = p.rows.pos0, top = p.bias_len - 1;
  const bool in_lds = p.bias_len <= SIG_BIAS_LDS;
  const float* bias = p.bias + (size_t)h * p.bias_len;
  const bf16_t* kb = (const bf16_t*)p.k_cache + ((size_t)p.rows.slot * p.kv_heads + g) * p.d.s64 * (DB * 64) + lane * 8;
  const bf16_t* vb = (const bf16_t*)p.v_cache + ((size_t)p.rows.slot * p.kv_heads + g) * p.d.s64 * p.d.vdim16 + lane * 8;
  const int MB16 = (p.M + 15) >> 4;
  uint4 qf[2][2 * DB];
  int qpos[2];
#pragma unroll
  for (int u = 0; u < 2; ++u) {
    qpos[u] = pos0 + min(q0 + 16 * u + l16, p.M - 1);
#pragma unroll
    for (int i = 0; i < 2 * DB; ++i)
      qf[u][i] = *reinterpret_cast<const uint4*>((const bf16_t*)p.q + h * p.q_z + ((size_t)min((q0 >> 4) + u, MB16 - 1) * DB * 2 + i) * 512 + lane * 8);
  }
  const int kend = pos0 + min(q0 + 31, p.M - 1) + 1;
  if (in_lds) {
    for (int k = tid; k < p.bias_len; k += 64 * SIGP_WAVES) lb[k] = bias[k] * -SIG_LOG2E;
    __syncthreads();
  }
  const float far = bias[top] * -SIG_LOG2E, c = -p.scale * SIG_LOG2E;
  tl_f32x4 acc[2][VT];
#pragma unroll
  for (int u = 0; u < 2; ++u)
#pragma unroll
    for (int d = 0; d < VT; ++d) acc[u][d] = tl_f32x4{0.f, 0.f, 0.f, 0.f};
  for (int k0 = 32 * wave; k0 < kend; k0 += 32 * SIGP_WAVES) {
    SigTile<DB, VT> t;
    t.load(kb, vb, k0, nvb);
    __builtin_amdgcn_sched_barrier(0);
#pragma unroll
    for (int u = 0; u < 2; ++u) {
      tl_f32x4 s[2];
      t.scores(qf[u], s);
      float w[8];
      const int near = pos0 + q0 + 16 * u - (k0 + 31);  // smallest distance of the tile
      if (near >= top) {  // uniform: every distance takes the last entry
#pragma unroll
        for (int e = 0; e < 8; ++e) w[e] = sig_weight(fmaf(s[e >> 2][e & 3], c, far));
      } else {
#pragma unroll
        for (int e = 0; e < 8; ++e) {
          const int n = qpos[u] - (k0 + 16 * (e >> 2) + 4 * kg + (e & 3)), i = min(max(n, 0), top);
          const float b = in_lds ? lb[i] : bias[i] * -SIG_LOG2E;
          w[e] = n >= 0 ? sig_weight(fmaf(s[e >> 2][e & 3], c, b)) : 0.f;
        }
      }
      t.add(w, acc[u]);
    }
  }
  const SigCols cols = sig_cols(p);
#pragma unroll
  for (int u = 0; u < 2; ++u) {
    if (u) __syncthreads();
#pragma unroll
    for (int d = 0; d < VT; ++d) *reinterpret_cast<tl_f32x4*>(&s_acc[wave][(d * 64 + lane) * 4]) = acc[u][d];
    __syncthreads();
    for (int sl = tid; sl < nvb * 64; sl += 64 * SIGP_WAVES) {
      const int d = sl >> 6, t = q0 + 16 * u + (sl & 15), k4 = (sl >> 4) & 3;
      if (t >= p.M) continue;
      tl_f32x4 o = *reinterpret_cast<const tl_f32x4*>(&s_acc[0][sl * 4]);
#pragma unroll
      for (int w = 1; w < SIGP_WAVES; ++w) o += *reinterpret_cast<const tl_f32x4*>(&s_acc[w][sl * 4]);
      const float f = 1.0f / (1.0f + expf(-bf2f(((const bf16_t*)p.raw)[(size_t)t * p.ld + cols.g + h])));
      const float r[4] = {o[0] * f, o[1] * f, o[2] * f, o[3] * f};
      Tl<bf16_t>::st4((bf16_t*)p.act + tl_off<bf16_t>(t, h * p.d.vdim16 + 16 * d + 4 * k4, p.d.out_k), r);
    }
  }
}

// ---- launchers ----
bool sig_step_fused(int dtype, const LmRows& rows, const vui_lm_dims& d) { return dtype == VUI_DTYPE_BF16 && !rows.seq && sig_mfma_ok(d); }
bool sig_mfma_ok(const vui_lm_dims& d) { return d.dim64 <= 256 && d.vdim16 <= 256; }

// pieces per row: as many workgroups as keep the chip busy
int sig_splits(int M, int heads, int kv_heads) {
  const int per = heads / kv_heads, wgs = M * kv_heads * ((per + 15) / 16);
  const int t = 1024 / wgs;
  return t < 1 ? 1 : (t > 64 ? 64 : t);
}

int launch_sig_prep(const SigAttnArgs& a, hipStream_t st) {
  const dim3 grid((a.heads + 2 * a.kv_heads + 3) / 4, a.M);
  if (a.dtype == VUI_DTYPE_F32) hipLaunchKernelGGL(sig_prep_kernel<float>, grid, dim3(256), 0, st, a);
  else hipLaunchKernelGGL(sig_prep_kernel<bf16_t>, grid, dim3(256), 0, st, a);
  HIP_TRY(hipGetLastError());
  return VUI_OK;
}

template <int DB, int VT>
static void piece_go(const SigAttnArgs& a, hipStream_t st) {
  const int per = a.heads / a.kv_heads;
  const dim3 grid(a.M, a.kv_heads * ((per + 15) / 16), a.n_splits);
  if (a.rows.seq) hipLaunchKernelGGL((sig_piece_mfma_kernel<DB, VT, false>), grid, dim3(256), 0, st, a);
  else hipLaunchKernelGGL((sig_piece_mfma_kernel<DB, VT, true>), grid, dim3(256), 0, st, a);
}
template <int DB, int VT>
static void prompt_go(const SigAttnArgs& a, hipStream_t st) {
  const size_t lds = a.bias_len <= SIG_BIAS_LDS ? (size_t)a.bias_len * 4 : 0;
  if (VT > 8)  // 64 KiB of accumulators beside the table
    (void)hipFuncSetAttribute((const void*)sig_prompt_kernel<DB, VT>, hipFuncAttributeMaxDynamicSharedMemorySize, SIG_BIAS_LDS * 4);
  hipLaunchKernelGGL((sig_prompt_kernel<DB, VT>), dim3((a.M + 31) / 32, a.heads), dim3(64 * SIGP_WAVES), lds, st, a);
}
#define SIG_DISPATCH(GO)                                                                              \
  switch (a.d.dim64 / 64) {                                                                           \
    case 1: SIG_VT(GO, 1) break;                                                                      \
    case 2: SIG_VT(GO, 2) break;                                                                      \
    case 3: SIG_VT(GO, 3) break;                                                                      \
    default: SIG_VT(GO, 4) break;                                                                     \
  }
#define SIG_VT(GO, DB)                                                                                \
  if (a.d.vdim16 <= 32) GO<DB, 2>(a, st);                                                             \
  else if (a.d.vdim16 <= 64) GO<DB, 4>(a, st);                                                        \
  else if (a.d.vdim16 <= 128) GO<DB, 8>(a, st);                                                       \
  else GO<DB, 16>(a, st);

int launch_sig_pieces(const SigAttnArgs& a, hipStream_t st) {
  if (a.n_splits < 1 || a.bias_len < 1 || a.heads % a.kv_heads) { vui_set_error("sigmoid attention: bad shape"); return VUI_EINVAL; }
  if (a.dtype == VUI_DTYPE_BF16 && sig_mfma_ok(a.d)) {
    SIG_DISPATCH(piece_go)
  } else {
    const dim3 grid(a.M, a.heads, a.n_splits);
    const size_t lds = (size_t)(a.d.dim64 + a.d.vdim16) * 4;
    if (a.dtype == VUI_DTYPE_F32) hipLaunchKernelGGL(sig_piece_kernel<float>, grid, dim3(256), lds, st, a);
    else hipLaunchKernelGGL(sig_piece_kernel<bf16_t>, grid, dim3(256), lds, st, a);
  }
  HIP_TRY(hipGetLastError());
  const dim3 grid((a.heads * a.d.vdim16 / 4 + 255) / 256, a.M);
  if (a.dtype == VUI_DTYPE_F32) hipLaunchKernelGGL(sig_merge_kernel<float>, grid, dim3(256), 0, st, a);
  else hipLaunchKernelGGL(sig_merge_kernel<bf16_t>, grid, dim3(256), 0, st, a);
  HIP_TRY(hipGetLastError());
  return VUI_OK;
}

int launch_sig_prompt(const SigAttnArgs& a, hipStream_t st) {
  if (!sig_mfma_ok(a.d) || a.dtype != VUI_DTYPE_BF16 || !a.rows.seq || a.bias_len < 1 || a.heads % a.kv_heads) { vui_set_error("sigmoid attention of a prompt: sizes out of range"); return VUI_EINVAL; }
  SIG_DISPATCH(prompt_go)
  HIP_TRY(hipGetLastError());
  return VUI_OK;
}
