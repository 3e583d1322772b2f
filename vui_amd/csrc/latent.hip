// Latent attention: per position the cache holds one normed latent c (kv_rank) and one rotated key part (rot_dim)
// common to the heads; head h's key is W_uk[h] c and its value W_uv[h] c.
//
// Two forms of the same sums.  Few rows attend in the latent space: the query goes through W_uk[h]^T once
// (latent_query_kernel), scores are its products with the cached latents, the softmax average of the latents goes
// through W_uv[h] (latent_value_kernel); nothing per key and head is ever formed.  Long blocks of a prompt expand
// keys and values of the whole slot once per layer (lm_gemm.hip) and run latent_prefill_kernel on them.
//
// Caches are tiled rows (tile.h), so that 16 keys x 64 latent columns are an operand of the matrix cores as they lie.
#include "common.h"
#include "lm.h"
#include "tile.h"

// ---- norm of the new latents and append; one wave per row ----
template <typename T>
__device__ __forceinline__ void latent_append_row(const LatentArgs& p, int m) {
  const int lane = threadIdx.x & 63;
  const float* src = p.craw + (size_t)m * p.d.rank16;
  float ss = 0.f;
  for (int k = lane * 4; k < p.d.rank16; k += 256) {  // columns beyond kv_rank hold zeros
    const float4 v = *reinterpret_cast<const float4*>(src + k);
    ss += (v.x * v.x + v.y * v.y) + (v.z * v.z + v.w * v.w);
  }
  ss = wave_sum(ss);
  const float r = 1.0f / sqrtf(ss / (float)p.rank + p.eps);
  const int slot = lm_slot(p.rows, m), pos = lm_pos(p.rows, m, slot);
  if (pos < 0 || pos >= p.rows.S) return;
  T* dst = (T*)p.c_cache + (size_t)slot * p.d.s64 * p.d.rank64;
  for (int k = lane * 4; k < p.d.rank16; k += 256) {
    const float4 v = *reinterpret_cast<const float4*>(src + k);
    const float4 w = *reinterpret_cast<const float4*>(p.latent_norm + k);
    const float o[4] = {v.x * r * w.x, v.y * r * w.y, v.z * r * w.z, v.w * r * w.w};
    Tl<T>::st4(dst + tl_off<T>(pos, k, p.d.rank64), o);
  }
}

template <typename T>
__global__ __launch_bounds__(256) void latent_append_kernel(const LatentArgs p) {
  const int m = blockIdx.x * 4 + (threadIdx.x >> 6);
  if (m < p.M) latent_append_row<T>(p, m);
}

// ---- queries into the latent space: qlat[h] (M x rank) = qu[h] (M x dim) W_uk[h]; a wave owns 16 latent columns ----
template <typename T>
__global__ __launch_bounds__(256) void latent_query_kernel(const LatentArgs p) {
  constexpr int EP = Tl<T>::EP, P = 16 / EP;
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), lane = threadIdx.x & 63;
  const int h = blockIdx.x, mt = blockIdx.z;
  if (h == p.heads) {  // the extra workgroups append the new latents
    for (int r = blockIdx.y * 4 + wave; r < 16; r += 4 * gridDim.y)
      if (mt * 16 + r < p.M) latent_append_row<T>(p, mt * 16 + r);
    return;
  }
  const int nb = blockIdx.y * 4 + wave;
  if (nb >= p.d.rank16 >> 4) return;
  const int nk = p.d.dim64 >> 6;
  const T* w = (const T*)p.w_uk_t + ((size_t)h * (p.d.rank16 >> 4) + nb) * nk * 1024 + lane * EP;
  const T* x = (const T*)p.qu + h * p.qu_z + (size_t)mt * nk * 1024 + lane * EP;
  tl_f32x4 acc = {0.f, 0.f, 0.f, 0.f};
  for (int k = 0; k < nk; ++k) {
    uint4 a[P], b[P];
#pragma unroll
    for (int i = 0; i < P; ++i) {
      a[i] = *reinterpret_cast<const uint4*>(w + (size_t)k * 1024 + 64 * EP * i);
      b[i] = *reinterpret_cast<const uint4*>(x + (size_t)k * 1024 + 64 * EP * i);
    }
#pragma unroll
    for (int i = 0; i < P; ++i) acc = Tl<T>::mma(a[i], b[i], acc);
  }
  const int m = mt * 16 + (lane & 15);
  if (m >= p.M) return;
  const float v[4] = {acc[0], acc[1], acc[2], acc[3]};
  Tl<T>::st4((T*)p.qlat + h * p.qlat_z + tl_off<T>(m, nb * 16 + 4 * (lane >> 4), p.d.rank64), v);
}

// A row that sees len keys is cut into pieces of this many (whole 32-key tiles), at most ns of them.  With more than
// four rows a piece has two tiles at least: there are pieces enough, and fewer are merged faster.
__device__ __forceinline__ int latent_chunk(int len, int ns, int M) { return max(((len + ns - 1) / ns + 31) & ~31, M > 4 ? 64 : 32); }
// keys [lo, hi) of piece sp
__device__ __forceinline__ void latent_range(int len, int ns, int M, int sp, int& lo, int& hi) {
  const int chunk = latent_chunk(len, ns, M);
  lo = min(sp * chunk, len);
  hi = min(lo + chunk, len);
}

// ---- attention in the latent space, any sizes: one workgroup per (row, head, split); fp32 arithmetic ----
#define LAT_TILE 256
#define LAT_ACC 8  // latent columns per thread: kv_rank up to 2048
template <typename T>
__global__ __launch_bounds__(256) void latent_attn_kernel(const LatentArgs p) {
  extern __shared__ __align__(16) float lq[];  // query: rank64 + rot32
  __shared__ float sc[LAT_TILE];
  __shared__ float red[4], red2[4];
  constexpr int EP = Tl<T>::EP;
  const int m = blockIdx.x, h = blockIdx.y, sp = blockIdx.z, tid = threadIdx.x, wave = tid >> 6, lane = tid & 63;
  const int R = p.d.rank64, RR = p.d.rot32;
  const int slot = lm_slot(p.rows, m);
  const int len = min(max(lm_pos(p.rows, m, slot) + 1, 1), p.rows.S);
  int lo, hi;
  latent_range(len, p.n_splits, p.M, sp, lo, hi);
  if (lo >= hi) return;  // no such piece: latent_value_kernel does not look for it
  for (int k = tid; k < R + RR; k += 256)
    lq[k] = k < R ? (k < p.d.rank16 ? El<T>::ld((const T*)p.qlat + h * p.qlat_z + tl_off<T>(m, k, R)) : 0.f)
                  : (k - R < p.d.rot16 ? El<T>::ld((const T*)p.qr + h * p.qr_z + tl_off<T, 32>(m, k - R, RR)) : 0.f);
  const T* cc = (const T*)p.c_cache + (size_t)slot * p.d.s64 * R;
  const T* kc = (const T*)p.kr_cache + (size_t)slot * p.d.s64 * RR;
  float acc[LAT_ACC];
#pragma unroll
  for (int i = 0; i < LAT_ACC; ++i) acc[i] = 0.f;
  float M = -INFINITY, L = 0.f;
  __syncthreads();
  for (int j0 = lo; j0 < hi; j0 += LAT_TILE) {
    const int j = j0 + tid, nj = min(LAT_TILE, hi - j0);
    float s = -INFINITY;
    if (j < hi) {
      float d = 0.f;
      for (int k = 0; k < R; k += EP) {
        const T* q = cc + tl_off<T>(j, k, R);
#pragma unroll
        for (int e = 0; e < EP; ++e) d = fmaf(lq[k + e], El<T>::ld(q + e), d);
      }
      for (int k = 0; k < RR; k += EP) {
        const T* q = kc + tl_off<T, 32>(j, k, RR);
#pragma unroll
        for (int e = 0; e < EP; ++e) d = fmaf(lq[R + k + e], El<T>::ld(q + e), d);
      }
      s = d * p.scale;
    }
    const float wm = wave_max(s);
    if (lane == 0) red[wave] = wm;
    __syncthreads();
    const float mn = fmaxf(M, fmaxf(fmaxf(red[0], red[1]), fmaxf(red[2], red[3])));
    const float e = j < hi ? expf(s - mn) : 0.f;
    sc[tid] = e;
    const float ws = wave_sum(e);
    if (lane == 0) red2[wave] = ws;
    __syncthreads();
    const float al = expf(M - mn);
    L = L * al + ((red2[0] + red2[1]) + (red2[2] + red2[3]));
    M = mn;
#pragma unroll
    for (int i = 0; i < LAT_ACC; ++i) {
      const int col = tid + 256 * i;
      if (col < R) {
        float a = acc[i] * al;
        for (int k = 0; k < nj; ++k) a = fmaf(sc[k], El<T>::ld(cc + tl_off<T>(j0 + k, col, R)), a);
        acc[i] = a;
      }
    }
    __syncthreads();
  }
  const size_t piece = ((size_t)m * p.heads + h) * p.n_splits + sp;
  if (tid == 0) *reinterpret_cast<float2*>(p.part_ml + 2 * piece) = make_float2(M, L);
#pragma unroll
  for (int i = 0; i < LAT_ACC; ++i)
    if (tid + 256 * i < R) p.part[piece * R + tid + 256 * i] = acc[i];
}

// ---- attention in the latent space on the matrix cores (bf16): one workgroup per (row, 16 heads, split) ----
// All heads read the same latents, so 32 keys are staged in LDS once and serve 16 heads.  Scores^T (keys x heads) =
// [c | k_rot] [q_lat | q_rot]^T, the four waves dealing key tile and half of the columns between them; every wave then
// has all scores of its lane's head and averages a quarter of the latent columns: out^T (columns x heads) = C^T p^T,
// the weights as a bf16 pair (value and remainder).  The transposed operand is gathered from LDS element by element.
// RK = rank64 / 64, RB = rot32 / 32.
template <int RK, int RB>
__global__ __launch_bounds__(256) void latent_attn_mfma_kernel(const LatentArgs p) {
  constexpr int CT = RK * 2048, RT = RB * 1024;  // elements of the staged tiles (32 keys)
  extern __shared__ __align__(16) bf16_t tile[];  // 2 x (CT + RT)
  __shared__ __align__(16) float sco[4][64 * 4];
  const int m = blockIdx.x, sp = blockIdx.z, tid = threadIdx.x;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6), lane = tid & 63, l16 = lane & 15, kg = lane >> 4;
  const int t = wave & 1, half = wave >> 1;
  const int head = blockIdx.y * 16 + l16, hq = min(head, p.heads - 1);
  const int slot = lm_slot(p.rows, m);
  const int len = min(max(lm_pos(p.rows, m, slot) + 1, 1), p.rows.S);
  int lo, hi;
  latent_range(len, p.n_splits, p.M, sp, lo, hi);
  const tl_u32x4* cc = reinterpret_cast<const tl_u32x4*>((const bf16_t*)p.c_cache + (size_t)slot * p.d.s64 * (RK * 64));
  const tl_u32x4* kc = reinterpret_cast<const tl_u32x4*>((const bf16_t*)p.kr_cache + (size_t)slot * p.d.s64 * (RB * 32));
  if (lo >= hi) return;  // no such piece
  // 32 keys are one contiguous run of either cache
  tl_u32x4 rc[RK], rr;
#define LAT_FETCH(j)                                                                            \
  {                                                                                             \
    const size_t jt = (size_t)((j) >> 5);                                                       \
    _Pragma("unroll") for (int i = 0; i < RK; ++i) rc[i] = cc[jt * (CT / 8) + tid + 256 * i];   \
    rr = kc[jt * (RT / 8) + min(tid, RT / 8 - 1)];                                              \
  }
#define LAT_STAGE(dst)                                                                          \
  {                                                                                             \
    tl_u32x4* sd = reinterpret_cast<tl_u32x4*>(dst);                                                  \
    _Pragma("unroll") for (int i = 0; i < RK; ++i) sd[tid + 256 * i] = rc[i];                   \
    if (tid < RT / 8) sd[CT / 8 + tid] = rr;                                                    \
  }
  LAT_FETCH(lo);
  // this wave's columns: piece `half` of every latent block, and a block of the rotated part (one wave pair without, RB = 1)
  const bool rot = RB == 2 || half == 0;
  uint4 qf[RK + 1];
  const int qrow = ((m & 15) + 16 * kg) * 8;
#pragma unroll
  for (int i = 0; i < RK; ++i)
    qf[i] = *reinterpret_cast<const uint4*>((const bf16_t*)p.qlat + hq * p.qlat_z + ((size_t)(m >> 4) * RK + i) * 1024 + half * 512 + qrow);
  qf[RK] = *reinterpret_cast<const uint4*>((const bf16_t*)p.qr + hq * p.qr_z + ((size_t)(m >> 4) * RB + (RB == 2 ? half : 0)) * 512 + qrow);
  tl_f32x4 acc[RK];
#pragma unroll
  for (int i = 0; i < RK; ++i) acc[i] = tl_f32x4{0.f, 0.f, 0.f, 0.f};
  float m_run = -INFINITY, l_run = 0.f;
  LAT_STAGE(tile);
  __syncthreads();
  int buf = 0;
  for (int j0 = lo; j0 < hi; j0 += 32) {
    const bf16_t* cur = tile + buf * (CT + RT);
    const bool more = j0 + 32 < hi;
    LAT_FETCH(more ? j0 + 32 : j0);
    tl_f32x4 s = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int i = 0; i < RK; ++i) s = Tl<bf16_t>::mma(*reinterpret_cast<const uint4*>(cur + (t * RK + i) * 1024 + half * 512 + lane * 8), qf[i], s);
    if (rot)  // uniform over the wave
      s = Tl<bf16_t>::mma(*reinterpret_cast<const uint4*>(cur + CT + (t * RB + (RB == 2 ? half : 0)) * 512 + lane * 8), qf[RK], s);
    *reinterpret_cast<tl_f32x4*>(&sco[half * 2 + t][lane * 4]) = s;
    __syncthreads();
    // keys j0 + 16 u + 4 kg + r of this lane's head
    float sv[8], mx = -INFINITY;
#pragma unroll
    for (int u = 0; u < 2; ++u) {
      const tl_f32x4 a = *reinterpret_cast<const tl_f32x4*>(&sco[u][lane * 4]) + *reinterpret_cast<const tl_f32x4*>(&sco[2 + u][lane * 4]);
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const float v = j0 + 16 * u + 4 * kg + r < hi ? a[r] * p.scale : -INFINITY;
        sv[4 * u + r] = v;
        mx = fmaxf(mx, v);
      }
    }
    mx = rows_max(mx);
    const float m_new = fmaxf(m_run, mx);  // finite: key j0 is in range
    const float alpha = expf(m_run - m_new);
    float pv[8], ps = 0.f;
#pragma unroll
    for (int e = 0; e < 8; ++e) { pv[e] = expf(sv[e] - m_new); ps += pv[e]; }
    l_run = l_run * alpha + ps;
    m_run = m_new;
    uint4 hi4, lo4;
    hi4.x = f2bf2(pv[0], pv[1]); hi4.y = f2bf2(pv[2], pv[3]); hi4.z = f2bf2(pv[4], pv[5]); hi4.w = f2bf2(pv[6], pv[7]);
    lo4.x = f2bf2(pv[0] - bf_lo(hi4.x), pv[1] - bf_hi(hi4.x)); lo4.y = f2bf2(pv[2] - bf_lo(hi4.y), pv[3] - bf_hi(hi4.y));
    lo4.z = f2bf2(pv[4] - bf_lo(hi4.z), pv[5] - bf_hi(hi4.z)); lo4.w = f2bf2(pv[6] - bf_lo(hi4.w), pv[7] - bf_hi(hi4.w));
#pragma unroll
    for (int i = 0; i < RK; ++i) {
      // 16 columns of block i, column group `wave`: column l16, the lane's eight keys
      const bf16_t* q = cur + i * 1024 + (l16 >> 3) * 512 + (4 * kg + 16 * wave) * 8 + (l16 & 7);
      uint4 v;
      v.x = (uint32_t)q[0] | ((uint32_t)q[8] << 16);
      v.y = (uint32_t)q[16] | ((uint32_t)q[24] << 16);
      const bf16_t* q1 = q + RK * 1024;
      v.z = (uint32_t)q1[0] | ((uint32_t)q1[8] << 16);
      v.w = (uint32_t)q1[16] | ((uint32_t)q1[24] << 16);
#pragma unroll
      for (int r = 0; r < 4; ++r) acc[i][r] *= alpha;
      acc[i] = Tl<bf16_t>::mma(v, hi4, acc[i]);
      acc[i] = Tl<bf16_t>::mma(v, lo4, acc[i]);
    }
    if (more) LAT_STAGE(tile + (buf ^ 1) * (CT + RT));
    __syncthreads();
    buf ^= 1;
  }
  l_run = rows_sum(l_run);
  if (head >= p.heads) return;
  const size_t piece = ((size_t)m * p.heads + head) * p.n_splits + sp;
  if (wave == 0 && kg == 0) *reinterpret_cast<float2*>(p.part_ml + 2 * piece) = make_float2(m_run, l_run);
#pragma unroll
  for (int i = 0; i < RK; ++i)
    *reinterpret_cast<tl_f32x4*>(p.part + piece * (RK * 64) + i * 64 + wave * 16 + 4 * kg) = acc[i];
}

// ---- merge of the pieces, value expansion through W_uv[h], head gate: up to 16 rows x 128 value dims of one head ----
template <typename T>
__global__ __launch_bounds__(512) void latent_value_kernel(const LatentArgs p, int rpw) {
  extern __shared__ __align__(16) unsigned char lv_raw[];
  T* xs = (T*)lv_raw;  // 16 x rank64, tiled
  constexpr int EP = Tl<T>::EP, P = 16 / EP, PRE = sizeof(T) == 2 ? 8 : 4;
  const int wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), lane = threadIdx.x & 63;
  const int h = blockIdx.x, m0 = blockIdx.z * rpw, R = p.d.rank64, ns = p.n_splits, nk = R >> 6;
  const int nb = blockIdx.y * 8 + wave, nvb = p.d.vdim16 >> 4;
  const int nrow = min(rpw, p.M - m0);
  const float gate = p.gate[(size_t)min(m0 + (lane & 15), p.M - 1) * p.d.heads16 + h];
  // the first weights are requested ahead of the merge
  const T* wv = (const T*)p.w_uv + ((size_t)h * nvb + min(nb, nvb - 1)) * nk * 1024 + lane * EP;
  uint4 wp[PRE][P];
#pragma unroll
  for (int k = 0; k < PRE; ++k)
#pragma unroll
    for (int i = 0; i < P; ++i) wp[k][i] = *reinterpret_cast<const uint4*>(wv + (size_t)min(k, nk - 1) * 1024 + 64 * EP * i);
  for (int it = wave; it < nrow * nk; it += 8) {  // a wave merges 64 columns of a row
    const int r = it / nk, k = (it - r * nk) * 64 + lane;
    const int m = m0 + r, slot = lm_slot(p.rows, m);
    const int len = min(max(lm_pos(p.rows, m, slot) + 1, 1), p.rows.S);
    const int chunk = latent_chunk(len, ns, p.M), np = (len + chunk - 1) / chunk;  // pieces that exist
    const size_t piece = ((size_t)m * p.heads + h) * ns;
    const float2 ml = *reinterpret_cast<const float2*>(p.part_ml + 2 * (piece + min(lane, np - 1)));
    const float* pc = p.part + piece * R + k;
    float v[16];  // sixteen loads in flight; a piece beyond the last gets weight zero
#pragma unroll
    for (int u = 0; u < 16; ++u) v[u] = pc[(size_t)min(u, np - 1) * R];
    const float M = wave_max(lane < np ? ml.x : -INFINITY);
    float w = lane < np ? expf(ml.x - M) : 0.f;
    w /= wave_sum(w * ml.y);
    float o = 0.f;
    for (int s0 = 0;;) {
#pragma unroll
      for (int u = 0; u < 16; ++u) o = fmaf(lane_f(w, min(s0 + u, 63)), s0 + u < np ? v[u] : 0.f, o);
      s0 += 16;
      if (s0 >= np) break;
#pragma unroll
      for (int u = 0; u < 16; ++u) v[u] = pc[(size_t)min(s0 + u, np - 1) * R];
    }
    El<T>::st(xs + tl_off<T>(r, k, R), o);
  }
  // rows without a position: their products are dropped, but must be numbers
  for (int i = threadIdx.x; i < (16 - nrow) * (R / 4); i += 512) {
    const float z[4] = {0.f, 0.f, 0.f, 0.f};
    Tl<T>::st4(xs + tl_off<T>(nrow + i / (R / 4), (i % (R / 4)) * 4, R), z);
  }
  __syncthreads();
  if (nb >= nvb) return;
  tl_f32x4 acc = {0.f, 0.f, 0.f, 0.f};
  auto step = [&](int k, const uint4* a) {
#pragma unroll
    for (int i = 0; i < P; ++i)
      acc = Tl<T>::mma(a[i], *reinterpret_cast<const uint4*>(xs + (size_t)k * 1024 + 64 * EP * i + lane * EP), acc);
  };
#pragma unroll
  for (int k = 0; k < PRE; ++k)
    if (k < nk) step(k, wp[k]);
  for (int k = PRE; k < nk; ++k) {
    uint4 a[P];
#pragma unroll
    for (int i = 0; i < P; ++i) a[i] = *reinterpret_cast<const uint4*>(wv + (size_t)k * 1024 + 64 * EP * i);
    step(k, a);
  }
  const int m = m0 + (lane & 15);
  if ((lane & 15) >= nrow) return;
  const float v[4] = {acc[0] * gate, acc[1] * gate, acc[2] * gate, acc[3] * gate};
  Tl<T>::st4((T*)p.act + tl_off<T>(m, h * p.d.vdim16 + nb * 16 + 4 * (lane >> 4), p.d.out_k), v);
}

// ---- expanded form for long blocks of one sequence (bf16): one workgroup per 16 queries and head ----
// Waves take 32 keys at a time in turn.  Scores^T (keys x queries) = K q^T leave a lane with eight keys of one query,
// which is operand layout for out^T = V^T p^T; the fp32 weights go in as a bf16 pair (value and remainder), so the
// average keeps about 16 bits of them.  DB = dim64 / 64, RB = rot32 / 32, VT >= vdim16 / 16.
#define LPF_WAVES (VT <= 4 ? 8 : 4)
template <int DB, int RB, int VT>
__global__ __launch_bounds__(64 * LPF_WAVES) void latent_prefill_kernel(const LatentArgs p) {
  __shared__ __align__(16) float s_acc[LPF_WAVES][VT * 256];
  __shared__ float s_m[LPF_WAVES][16], s_l[LPF_WAVES][16];
  const int tid = threadIdx.x, wave = __builtin_amdgcn_readfirstlane(tid >> 6), lane = tid & 63;
  const int l16 = lane & 15, kg = lane >> 4;
  const int qt = gridDim.x - 1 - blockIdx.x, h = blockIdx.y;  // the tiles with the most keys start first
  const int q0 = qt * 16, T = p.M, pos0 = p.rows.pos0;
  const int nvb = p.d.vdim16 >> 4;
  const int qlast = pos0 + min(q0 + l16, T - 1);  // last visible key of this lane's query
  const int kend = pos0 + min(q0 + 15, T - 1) + 1;
  const bf16_t* qu = (const bf16_t*)p.qu + h * p.qu_z + (size_t)qt * DB * 1024 + lane * 8;
  const bf16_t* qr = (const bf16_t*)p.qr + h * p.qr_z + (size_t)qt * RB * 512 + lane * 8;
  uint4 qf[2 * DB + RB];
#pragma unroll
  for (int i = 0; i < 2 * DB; ++i) qf[i] = *reinterpret_cast<const uint4*>(qu + i * 512);
#pragma unroll
  for (int i = 0; i < RB; ++i) qf[2 * DB + i] = *reinterpret_cast<const uint4*>(qr + i * 512);
  const bf16_t* kb = (const bf16_t*)p.kx + h * p.kx_z + lane * 8;
  const bf16_t* rb = (const bf16_t*)p.kr_cache + (size_t)p.rows.slot * p.d.s64 * (RB * 32) + lane * 8;
  const bf16_t* vb = (const bf16_t*)p.vx + h * p.vx_z + lane * 8;
  const int vstep = (p.d.s64 >> 5) * 512;

  tl_f32x4 acc[VT];
#pragma unroll
  for (int d = 0; d < VT; ++d) acc[d] = tl_f32x4{0.f, 0.f, 0.f, 0.f};
  float m_run = -INFINITY, l_run = 0.f;
  for (int k0 = 32 * wave; k0 < kend; k0 += 32 * LPF_WAVES) {
    uint4 kf[2][2 * DB + RB], vf[VT];
#pragma unroll
    for (int t = 0; t < 2; ++t) {
#pragma unroll
      for (int i = 0; i < 2 * DB; ++i) kf[t][i] = *reinterpret_cast<const uint4*>(kb + (size_t)((k0 >> 4) + t) * DB * 1024 + i * 512);
#pragma unroll
      for (int i = 0; i < RB; ++i) kf[t][2 * DB + i] = *reinterpret_cast<const uint4*>(rb + (size_t)((k0 >> 4) + t) * RB * 512 + i * 512);
    }
#pragma unroll
    for (int d = 0; d < VT; ++d) vf[d] = *reinterpret_cast<const uint4*>(vb + (size_t)min(d, nvb - 1) * vstep + (size_t)(k0 >> 5) * 512);
    __builtin_amdgcn_sched_barrier(0);
    tl_f32x4 sc[2];
#pragma unroll
    for (int t = 0; t < 2; ++t) {
      sc[t] = tl_f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int i = 0; i < 2 * DB + RB; ++i) sc[t] = Tl<bf16_t>::mma(kf[t][i], qf[i], sc[t]);
    }
    float sv[8], mx = -INFINITY;
#pragma unroll
    for (int t = 0; t < 2; ++t)
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const int j = k0 + 16 * t + 4 * kg + r;
        const float v = j <= qlast ? sc[t][r] * p.scale : -INFINITY;
        sv[4 * t + r] = v;
        mx = fmaxf(mx, v);
      }
    mx = rows_max(mx);
    const float m_new = fmaxf(m_run, mx);
    const float m_use = m_new == -INFINITY ? 0.f : m_new;
    const float alpha = expf(m_run - m_use);
    float pv[8], lo[8], ps = 0.f;
    uint4 hi4, lo4;
#pragma unroll
    for (int e = 0; e < 8; ++e) { pv[e] = expf(sv[e] - m_use); ps += pv[e]; }
    l_run = l_run * alpha + ps;
    m_run = m_new;
    hi4.x = f2bf2(pv[0], pv[1]); hi4.y = f2bf2(pv[2], pv[3]); hi4.z = f2bf2(pv[4], pv[5]); hi4.w = f2bf2(pv[6], pv[7]);
    lo[0] = pv[0] - bf_lo(hi4.x); lo[1] = pv[1] - bf_hi(hi4.x); lo[2] = pv[2] - bf_lo(hi4.y); lo[3] = pv[3] - bf_hi(hi4.y);
    lo[4] = pv[4] - bf_lo(hi4.z); lo[5] = pv[5] - bf_hi(hi4.z); lo[6] = pv[6] - bf_lo(hi4.w); lo[7] = pv[7] - bf_hi(hi4.w);
    lo4.x = f2bf2(lo[0], lo[1]); lo4.y = f2bf2(lo[2], lo[3]); lo4.z = f2bf2(lo[4], lo[5]); lo4.w = f2bf2(lo[6], lo[7]);
#pragma unroll
    for (int d = 0; d < VT; ++d) {
#pragma unroll
      for (int r = 0; r < 4; ++r) acc[d][r] *= alpha;
      acc[d] = Tl<bf16_t>::mma(vf[d], hi4, acc[d]);
      acc[d] = Tl<bf16_t>::mma(vf[d], lo4, acc[d]);
    }
  }
  l_run = rows_sum(l_run);
  if (kg == 0) { s_m[wave][l16] = m_run; s_l[wave][l16] = l_run; }
#pragma unroll
  for (int d = 0; d < VT; ++d) *reinterpret_cast<tl_f32x4*>(&s_acc[wave][(d * 64 + lane) * 4]) = acc[d];
  __syncthreads();
  for (int sl = tid; sl < nvb * 64; sl += 64 * LPF_WAVES) {
    const int d = sl >> 6, ln = sl & 63, q = ln & 15, g4 = ln >> 4;
    const int t = q0 + q;
    if (t >= T) continue;
    float M = -INFINITY;
#pragma unroll
    for (int w = 0; w < LPF_WAVES; ++w) M = fmaxf(M, s_m[w][q]);
    float den = 0.f, o[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int w = 0; w < LPF_WAVES; ++w) {
      const float f = s_m[w][q] == -INFINITY ? 0.f : expf(s_m[w][q] - M);
      den = fmaf(f, s_l[w][q], den);
#pragma unroll
      for (int r = 0; r < 4; ++r) o[r] = fmaf(f, s_acc[w][sl * 4 + r], o[r]);
    }
    const float inv = p.gate[(size_t)t * p.d.heads16 + h] / den;
#pragma unroll
    for (int r = 0; r < 4; ++r) o[r] *= inv;
    Tl<bf16_t>::st4((bf16_t*)p.act + tl_off<bf16_t>(t, h * p.d.vdim16 + 16 * d + 4 * g4, p.d.out_k), o);
  }
}

// ---- launchers ----
int launch_latent_append(const LatentArgs& a, hipStream_t st) {
  if (a.dtype == VUI_DTYPE_F32) hipLaunchKernelGGL(latent_append_kernel<float>, dim3((a.M + 3) / 4), dim3(256), 0, st, a);
  else hipLaunchKernelGGL(latent_append_kernel<bf16_t>, dim3((a.M + 3) / 4), dim3(256), 0, st, a);
  HIP_TRY(hipGetLastError());
  return VUI_OK;
}

int launch_latent_query(const LatentArgs& a, hipStream_t st) {
  const dim3 grid(a.heads + (a.own ? 1 : 0), (a.d.rank16 / 16 + 3) / 4, (a.M + 15) / 16);
  if (a.dtype == VUI_DTYPE_F32) hipLaunchKernelGGL(latent_query_kernel<float>, grid, dim3(256), 0, st, a);
  else hipLaunchKernelGGL(latent_query_kernel<bf16_t>, grid, dim3(256), 0, st, a);
  HIP_TRY(hipGetLastError());
  return VUI_OK;
}

bool latent_mfma_ok(const vui_lm_dims& d) { return d.rank64 <= 512 && d.rot32 <= 64; }

template <int RK, int RB>
static int lam_go(const LatentArgs& a, hipStream_t st) {
  constexpr int lds = 2 * (RK * 2048 + RB * 1024) * 2;
  if (lds > 60 * 1024) {
    static bool set = false;
    if (!set) {
      HIP_TRY(hipFuncSetAttribute((const void*)latent_attn_mfma_kernel<RK, RB>, hipFuncAttributeMaxDynamicSharedMemorySize, lds));
      set = true;
    }
  }
  hipLaunchKernelGGL((latent_attn_mfma_kernel<RK, RB>), dim3(a.M, (a.heads + 15) / 16, a.n_splits), dim3(256), lds, st, a);
  HIP_TRY(hipGetLastError());
  return VUI_OK;
}
template <int RB>
static int lam_rank(const LatentArgs& a, hipStream_t st) {
  switch (a.d.rank64 / 64) {
    case 1: return lam_go<1, RB>(a, st);
    case 2: return lam_go<2, RB>(a, st);
    case 3: return lam_go<3, RB>(a, st);
    case 4: return lam_go<4, RB>(a, st);
    case 5: return lam_go<5, RB>(a, st);
    case 6: return lam_go<6, RB>(a, st);
    case 7: return lam_go<7, RB>(a, st);
    default: return lam_go<8, RB>(a, st);
  }
}

int launch_latent_attn(const LatentArgs& a, hipStream_t st) {
  if (a.n_splits < 1 || a.n_splits > 64 || a.d.rank64 > 256 * LAT_ACC) { vui_set_error("latent attention: rank %d, splits %d out of range", a.d.rank64, a.n_splits); return VUI_EINVAL; }
  if (a.dtype == VUI_DTYPE_BF16 && latent_mfma_ok(a.d)) return a.d.rot32 == 32 ? lam_rank<1>(a, st) : lam_rank<2>(a, st);
  const dim3 grid(a.M, a.heads, a.n_splits);
  const size_t lds = (size_t)(a.d.rank64 + a.d.rot32) * 4;
  if (a.dtype == VUI_DTYPE_F32) hipLaunchKernelGGL(latent_attn_kernel<float>, grid, dim3(256), lds, st, a);
  else hipLaunchKernelGGL(latent_attn_kernel<bf16_t>, grid, dim3(256), lds, st, a);
  HIP_TRY(hipGetLastError());
  return VUI_OK;
}

int launch_latent_value(const LatentArgs& a, hipStream_t st) {
  // rows per workgroup: all 16 of a tile only when there are enough heads and rows to fill the chip without
  int rpw = 1;
  while (rpw < 16 && a.M * a.heads > 192 * rpw) rpw *= 2;
  const dim3 grid(a.heads, (a.d.vdim16 / 16 + 7) / 8, (a.M + rpw - 1) / rpw);
  const bool f32 = a.dtype == VUI_DTYPE_F32;
  const size_t lds = (size_t)16 * a.d.rank64 * (f32 ? 4 : 2);
  if (lds > 64 * 1024) {
    HIP_TRY(hipFuncSetAttribute(f32 ? (const void*)latent_value_kernel<float> : (const void*)latent_value_kernel<bf16_t>,
                                hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds));
  }
  if (f32) hipLaunchKernelGGL(latent_value_kernel<float>, grid, dim3(512), lds, st, a, rpw);
  else hipLaunchKernelGGL(latent_value_kernel<bf16_t>, grid, dim3(512), lds, st, a, rpw);
  HIP_TRY(hipGetLastError());
  return VUI_OK;
}

bool latent_expand_ok(const vui_lm_dims& d) { return d.dim64 <= 128 && d.rot32 <= 64 && d.vdim16 <= 128; }

template <int DB, int RB>
static void lpf_go(const LatentArgs& a, hipStream_t st) {
  const dim3 grid((a.M + 15) / 16, a.heads);
  if (a.d.vdim16 <= 32) hipLaunchKernelGGL((latent_prefill_kernel<DB, RB, 2>), grid, dim3(512), 0, st, a);
  else if (a.d.vdim16 <= 64) hipLaunchKernelGGL((latent_prefill_kernel<DB, RB, 4>), grid, dim3(512), 0, st, a);
  else hipLaunchKernelGGL((latent_prefill_kernel<DB, RB, 8>), grid, dim3(256), 0, st, a);
}
int launch_latent_prefill_attn(const LatentArgs& a, hipStream_t st) {
  if (!latent_expand_ok(a.d) || a.dtype != VUI_DTYPE_BF16 || !a.rows.seq) { vui_set_error("latent prefill: sizes out of range"); return VUI_EINVAL; }
  if (a.d.dim64 == 64) { if (a.d.rot32 == 32) lpf_go<1, 1>(a, st); else lpf_go<1, 2>(a, st); }
  else { if (a.d.rot32 == 32) lpf_go<2, 1>(a, st); else lpf_go<2, 2>(a, st); }
  HIP_TRY(hipGetLastError());
  return VUI_OK;
}
