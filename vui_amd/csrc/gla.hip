// Gated linear attention: per head S <- diag(a) S + k v^T and o = S^T q, where a decays every key channel (row of S) by
// a number of its own, a = sigmoid(W_a2 l + b)^(1 / tau) with l the low-rank part of the projection; o is normed over
// the value channels and multiplied by silu of a gate.  Decays, state and everything around it are fp32.
//
// Two forms.  gla_step_kernel walks positions one by one (decode steps, short portions, any sizes).  A longer portion
// goes by chunks of 32 positions with b_t the sum of the log decays inside the chunk:
//   chunk:  U = sum_s (k_s exp(b_end - b_s)) v_s^T, one workgroup per chunk and head;
//   carry:  the states between chunks, S <- diag(exp(b_end)) S + U;
//   read:   o_t = (q_t exp(b_t)) S + sum_(s <= t) (sum_d q_td k_sd exp(b_td - b_sd)) v_s.
// No exponent is ever positive: inside 16 positions the differences are formed one by one, between the halves of a chunk
// they are split at the border.  Products run on the fp32 matrix instructions.
#include "common.h"
#include "lm.h"
#include "tile.h"

struct GlaCols { int k, v, g, a; };
__device__ __forceinline__ GlaCols gla_cols(const GlaArgs& p) {
  GlaCols c;
  c.k = p.heads * p.d.dim16;
  c.v = c.k + p.heads * p.d.dim16;
  c.g = c.v + p.heads * p.d.vdim16;
  c.a = c.g + p.heads * p.d.vdim16;
  return c;
}

// log of the decay of channel d of head h: -softplus(-z) / tau; low: the row's low-rank part
template <typename T>
__device__ __forceinline__ float gla_log_decay(const GlaArgs& p, const T* low, int h, int d) {
  const float* w = p.w_a2 + ((size_t)h * p.d.dim16 + d) * p.rank;
  float z = p.a2_bias[h * p.d.dim16 + d];
  for (int r = 0; r < p.rank; ++r) z = fmaf(w[r], El<T>::ld(low + r), z);
  return -(fmaxf(-z, 0.f) + log1pf(expf(-fabsf(z)))) * p.inv_tau;
}

__device__ __forceinline__ float silu_exact(float v) { return v / (1.0f + expf(-v)); }

// ---- positions one by one; one workgroup per head and slot ----
#define GLA_THREADS 512
#define GLA_PRE 8
template <typename T>
__global__ __launch_bounds__(GLA_THREADS) void gla_step_kernel(const GlaArgs p) {
  extern __shared__ __align__(16) float gl[];  // decay, key, query (dim16 each), value (vdim16), sums (passes, vdim16)
  __shared__ float red[GLA_THREADS / 64];
  const int h = blockIdx.x, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int D = p.d.dim16, V = p.d.vdim16, vq = V >> 2, per = GLA_THREADS / vq;  // rows of S per pass
  float *la = gl, *lk = gl + D, *lq = gl + 2 * D, *lv = gl + 3 * D, *ls = lv + V;
  const GlaCols c = gla_cols(p);
  const int c4 = (tid % vq) * 4, r0 = tid / vq;
  const bool work = r0 < per;
  const int m0 = p.rows.seq ? 0 : blockIdx.y, m1 = p.rows.seq ? p.M : m0 + 1;
  const int slot = lm_slot(p.rows, m0);
  float* S = p.state + ((size_t)slot * p.heads + h) * D * V;
  for (int m = m0; m < m1; ++m) {
    const bool fresh = lm_pos(p.rows, m, slot) <= 0;
    tl_f32x4 s[GLA_PRE];  // the first rows are on their way while the decays are computed
#pragma unroll
    for (int i = 0; i < GLA_PRE; ++i) s[i] = *reinterpret_cast<const tl_f32x4*>(S + (size_t)min(r0 + i * per, D - 1) * V + c4);
    const T* row = (const T*)p.raw + (size_t)m * p.ld;
    for (int d = tid; d < D; d += GLA_THREADS) {
      la[d] = expf(gla_log_decay<T>(p, row + c.a, h, d));
      lk[d] = El<T>::ld(row + c.k + h * D + d);
      lq[d] = El<T>::ld(row + h * D + d) * p.q_scale;
    }
    for (int d = tid; d < V; d += GLA_THREADS) lv[d] = El<T>::ld(row + c.v + h * V + d);
    __syncthreads();
    tl_f32x4 o = {0.f, 0.f, 0.f, 0.f};
    if (work) {
      const tl_f32x4 v = *reinterpret_cast<const tl_f32x4*>(lv + c4);
      for (int base = r0;;) {
#pragma unroll
        for (int i = 0; i < GLA_PRE; ++i) {
          const int d = base + i * per;
          if (d < D) {
            const float a = fresh ? 0.f : la[d], k = lk[d], q = lq[d];
            tl_f32x4 n;
#pragma unroll
            for (int e = 0; e < 4; ++e) {
              n[e] = fresh ? k * v[e] : fmaf(a, s[i][e], k * v[e]);
              o[e] = fmaf(q, n[e], o[e]);
            }
            *reinterpret_cast<tl_f32x4*>(S + (size_t)d * V + c4) = n;
          }
        }
        base += GLA_PRE * per;
        if (base >= D) break;
#pragma unroll
        for (int i = 0; i < GLA_PRE; ++i) s[i] = *reinterpret_cast<const tl_f32x4*>(S + (size_t)min(base + i * per, D - 1) * V + c4);
      }
      *reinterpret_cast<tl_f32x4*>(ls + r0 * V + c4) = o;
    }
    __syncthreads();
    float ss = 0.f;
    for (int d = tid; d < V; d += GLA_THREADS) {
      float t = 0.f;
      for (int r = 0; r < per; ++r) t += ls[r * V + d];
      ls[d] = t;  // row 0 is this thread's own column
      ss = fmaf(t, t, ss);
    }
    ss = wave_sum(ss);
    if (lane == 0) red[wave] = ss;
    __syncthreads();
    float t = 0.f;
#pragma unroll
    for (int w = 0; w < GLA_THREADS / 64; ++w) t += red[w];
    const float r = 1.0f / sqrtf(t / (float)p.vdim + p.eps);
    for (int d = tid; d < V; d += GLA_THREADS)
      El<T>::st((T*)p.act + tl_off<T>(m, h * V + d, p.d.out_k), ls[d] * r * p.head_norm[d] * silu_exact(El<T>::ld(row + c.g + h * V + d)));
    if (m + 1 < m1) {
      __threadfence_block();
      __syncthreads();
    }
  }
}

// ---- chunk: log decays, their sums, and what the chunk adds to the state ----
// LDS rows are D + 1 long: 16 rows at one column fall into different banks.
#define GC LM_GLA_CHUNK
template <typename T>
__global__ __launch_bounds__(256) void gla_chunk_kernel(const GlaArgs p) {
  extern __shared__ __align__(16) float gl[];  // b, then decayed keys (GC, D + 1); values (GC, V + 1); low-rank parts (GC, rank)
  const int ck = blockIdx.x, h = blockIdx.y, tid = threadIdx.x, lane = tid & 63, l16 = lane & 15, kg = lane >> 4;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int D = p.d.dim16, V = p.d.vdim16, DS = D + 1, VS = V + 1, t0 = ck * GC, n = min(GC, p.M - t0);
  float *lb = gl, *lv = gl + GC * DS;
  T* low = (T*)(lv + GC * VS);
  const GlaCols c = gla_cols(p);
  const T* raw = (const T*)p.raw + (size_t)t0 * p.ld;
  for (int i = tid; i < n * p.rank; i += 256) low[i] = raw[(size_t)(i / p.rank) * p.ld + c.a + i % p.rank];
  for (int i = tid; i < GC * V; i += 256) {
    const int t = i / V, d = i - t * V;
    lv[t * VS + d] = t < n ? El<T>::ld(raw + (size_t)t * p.ld + c.v + h * V + d) : 0.f;
  }
  __syncthreads();
  for (int i = tid; i < n * D; i += 256) {
    const int t = i / D, d = i - t * D;
    lb[t * DS + d] = gla_log_decay<T>(p, low + t * p.rank, h, d);
  }
  __syncthreads();
  for (int d = tid; d < D; d += 256) {
    float b = 0.f;
    for (int t = 0; t < n; ++t) {
      b += lb[t * DS + d];
      lb[t * DS + d] = b;
      p.bsum[((size_t)(t0 + t) * p.heads + h) * D + d] = b;
    }
    p.dec[((size_t)ck * p.heads + h) * D + d] = expf(b);
    for (int t = 0; t < GC; ++t)  // positions beyond the portion add nothing
      lb[t * DS + d] = t < n ? El<T>::ld(raw + (size_t)t * p.ld + c.k + h * D + d) * expf(b - lb[t * DS + d]) : 0.f;
  }
  __syncthreads();
  float* U = p.upd + ((size_t)ck * p.heads + h) * D * V;
  const int nv = V >> 4, tiles = (D >> 4) * nv;
  for (int i = wave; i < tiles; i += 4) {
    const int dt = i / nv, vt = i - dt * nv;
    tl_f32x4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int s = 0; s < GC; s += 4)
      acc = __builtin_amdgcn_mfma_f32_16x16x4f32(lv[(s + kg) * VS + vt * 16 + l16], lb[(s + kg) * DS + dt * 16 + l16], acc, 0, 0, 0);
    *reinterpret_cast<tl_f32x4*>(U + (size_t)(dt * 16 + l16) * V + vt * 16 + 4 * kg) = acc;
  }
}

// ---- carry: what a chunk adds is replaced by the state it starts from ----
__global__ __launch_bounds__(256) void gla_carry_kernel(const GlaArgs p, int nchunks) {
  const int per = p.d.dim16 * p.d.vdim16 / 4, i = blockIdx.x * 256 + threadIdx.x;  // four value channels of a row of S
  if (i >= per * p.heads) return;
  const int h = i / per, e = (i - h * per) * 4, d = e / p.d.vdim16;
  const size_t size = (size_t)per * 4, step = size * p.heads;
  float* S = p.state + (size_t)p.rows.slot * step + h * size + e;
  float* U = p.upd + h * size + e;
  const float* dec = p.dec + h * p.d.dim16 + d;
  tl_f32x4 s = {0.f, 0.f, 0.f, 0.f};
  if (p.rows.pos0 > 0) s = *reinterpret_cast<const tl_f32x4*>(S);
  for (int c0 = 0; c0 < nchunks; c0 += 8) {
    tl_f32x4 u[8];
    float a[8];
#pragma unroll
    for (int k = 0; k < 8; ++k) {
      const int c = min(c0 + k, nchunks - 1);
      u[k] = *reinterpret_cast<const tl_f32x4*>(U + c * step);
      a[k] = dec[(size_t)c * p.heads * p.d.dim16];
    }
#pragma unroll
    for (int k = 0; k < 8; ++k)
      if (c0 + k < nchunks) {
        *reinterpret_cast<tl_f32x4*>(U + (size_t)(c0 + k) * step) = s;
#pragma unroll
        for (int r = 0; r < 4; ++r) s[r] = fmaf(a[k], s[r], u[k][r]);
      }
  }
  *reinterpret_cast<tl_f32x4*>(S) = s;
}

// ---- read: outputs of a chunk; waves = 2 halves of the positions x 2 sets of value tiles (NV each) ----
template <typename T, int NV>
__global__ __launch_bounds__(256) void gla_read_kernel(const GlaArgs p) {
  extern __shared__ __align__(16) float gl[];  // b, q, k (GC, D + 1)
  __shared__ float A[GC][GC + 1], half[4][16][17], red[2][2][16];
  const int ck = blockIdx.x, h = blockIdx.y, tid = threadIdx.x, lane = tid & 63, l16 = lane & 15, kg = lane >> 4;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int D = p.d.dim16, V = p.d.vdim16, DS = D + 1, t0 = ck * GC, n = min(GC, p.M - t0), nv = V >> 4;
  float *lb = gl, *lq = gl + GC * DS, *lk = gl + 2 * GC * DS;
  const GlaCols c = gla_cols(p);
  const T* raw = (const T*)p.raw + (size_t)t0 * p.ld;
  for (int i = tid; i < GC * D; i += 256) {
    const int t = i / D, d = i - t * D;
    const bool live = t < n;
    lb[t * DS + d] = live ? p.bsum[((size_t)(t0 + t) * p.heads + h) * D + d] : 0.f;
    lq[t * DS + d] = live ? El<T>::ld(raw + (size_t)t * p.ld + h * D + d) * p.q_scale : 0.f;
    lk[t * DS + d] = live ? El<T>::ld(raw + (size_t)t * p.ld + c.k + h * D + d) : 0.f;
  }
  __syncthreads();
  {  // the two triangles of 16 positions
    const int o = (tid >> 7) * 16, s = o + (tid & 15);
#pragma unroll
    for (int u = 0; u < 2; ++u) {
      const int t = o + ((tid >> 4) & 7) + 8 * u;
      float a = 0.f;
      if (s <= t && t < n) {
        const float *q = lq + t * DS, *bt = lb + t * DS, *k = lk + s * DS, *bs = lb + s * DS;
        for (int d = 0; d < D; ++d) a = fmaf(q[d] * k[d], sizeof(T) == 4 ? expf(bt[d] - bs[d]) : __expf(bt[d] - bs[d]), a);
      }
      A[t][s] = a;
    }
  }
  {  // later half on earlier half: a wave sums a quarter of the channels
    tl_f32x4 acc = {0.f, 0.f, 0.f, 0.f};
    const int d1 = D * (wave + 1) / 4;
    for (int d0 = D * wave / 4; d0 < d1; d0 += 4) {
      const int d = d0 + kg;
      const float e = lb[15 * DS + d];
      const bool later = 16 + l16 < n;
      const float kk = lk[l16 * DS + d] * expf(n > 15 ? e - lb[l16 * DS + d] : 0.f);
      const float qq = later ? lq[(16 + l16) * DS + d] * expf(lb[(16 + l16) * DS + d] - e) : 0.f;
      acc = __builtin_amdgcn_mfma_f32_16x16x4f32(kk, qq, acc, 0, 0, 0);
    }
#pragma unroll
    for (int r = 0; r < 4; ++r) half[wave][l16][4 * kg + r] = acc[r];  // [later][earlier]
  }
  __syncthreads();
  {
    const int t = tid >> 4, s = tid & 15;
    A[16 + t][s] = (half[0][t][s] + half[1][t][s]) + (half[2][t][s] + half[3][t][s]);
    A[s][16 + t] = 0.f;
  }
  for (int i = tid; i < GC * D; i += 256) {
    const int t = i / D, d = i - t * D;
    lq[t * DS + d] *= expf(lb[t * DS + d]);
  }
  __syncthreads();
  const int th = wave & 1, vs = wave >> 1, t = th * 16 + l16;
  const float* S = p.upd + ((size_t)ck * p.heads + h) * D * V;
  tl_f32x4 acc[NV];
#pragma unroll
  for (int i = 0; i < NV; ++i) acc[i] = tl_f32x4{0.f, 0.f, 0.f, 0.f};
  if (ck > 0 || p.rows.pos0 > 0) {
    for (int d0 = 0; d0 < D; d0 += 16) {
      float q[4], sv[4][NV];
#pragma unroll
      for (int u = 0; u < 4; ++u) {
        q[u] = lq[t * DS + d0 + 4 * u + kg];
#pragma unroll
        for (int i = 0; i < NV; ++i) sv[u][i] = S[(size_t)(d0 + 4 * u + kg) * V + min(vs + 2 * i, nv - 1) * 16 + l16];
      }
#pragma unroll
      for (int u = 0; u < 4; ++u)
#pragma unroll
        for (int i = 0; i < NV; ++i) acc[i] = __builtin_amdgcn_mfma_f32_16x16x4f32(sv[u][i], q[u], acc[i], 0, 0, 0);
    }
  }
#pragma unroll
  for (int s0 = 0; s0 < GC; s0 += 4) {
    const int s = s0 + kg;
    const float a = A[t][s];
    const T* v = raw + (size_t)min(s, n - 1) * p.ld + c.v + h * V + l16;
#pragma unroll
    for (int i = 0; i < NV; ++i) acc[i] = __builtin_amdgcn_mfma_f32_16x16x4f32(El<T>::ld(v + min(vs + 2 * i, nv - 1) * 16), a, acc[i], 0, 0, 0);
  }
  float ss = 0.f;
#pragma unroll
  for (int i = 0; i < NV; ++i)
    if (vs + 2 * i < nv)
#pragma unroll
      for (int r = 0; r < 4; ++r) ss = fmaf(acc[i][r], acc[i][r], ss);
  ss = rows_sum(ss);
  if (kg == 0) red[vs][th][l16] = ss;
  __syncthreads();
  const float r = 1.0f / sqrtf((red[0][th][l16] + red[1][th][l16]) / (float)p.vdim + p.eps);
  if (t >= n) return;
#pragma unroll
  for (int i = 0; i < NV; ++i) {
    const int v0 = (vs + 2 * i) * 16 + 4 * kg;
    if (vs + 2 * i >= nv) continue;
    float o[4];
#pragma unroll
    for (int e = 0; e < 4; ++e)
      o[e] = acc[i][e] * r * p.head_norm[v0 + e] * silu_exact(El<T>::ld(raw + (size_t)t * p.ld + c.g + h * V + v0 + e));
    Tl<T>::st4((T*)p.act + tl_off<T>(t0 + t, h * V + v0, p.d.out_k), o);
  }
}

// ---- launchers ----
static int lds_attr(const void* f, size_t bytes) {
  if (bytes > 40 * 1024) HIP_TRY(hipFuncSetAttribute(f, hipFuncAttributeMaxDynamicSharedMemorySize, (int)bytes));
  return VUI_OK;
}

int launch_gla_step(const GlaArgs& a, hipStream_t st) {
  const int per = a.d.vdim16 ? GLA_THREADS / (a.d.vdim16 >> 2) : 0;
  if (per < 1) { vui_set_error("gated linear attention: value size %d too large", a.vdim); return VUI_EINVAL; }
  const size_t lds = (size_t)(3 * a.d.dim16 + (1 + per) * a.d.vdim16) * 4;
  const dim3 grid(a.heads, a.rows.seq ? 1 : a.M);
  int rc;
  if (a.dtype == VUI_DTYPE_F32) {
    if ((rc = lds_attr((const void*)gla_step_kernel<float>, lds))) return rc;
    hipLaunchKernelGGL(gla_step_kernel<float>, grid, dim3(GLA_THREADS), lds, st, a);
  } else {
    if ((rc = lds_attr((const void*)gla_step_kernel<bf16_t>, lds))) return rc;
    hipLaunchKernelGGL(gla_step_kernel<bf16_t>, grid, dim3(GLA_THREADS), lds, st, a);
  }
  HIP_TRY(hipGetLastError());
  return VUI_OK;
}

bool gla_chunk_ok(const vui_lm_dims& d) { return d.dim16 <= 256 && d.vdim16 <= 256; }

template <typename T, int NV>
static int read_go(const GlaArgs& a, int nchunks, hipStream_t st) {
  const size_t lds = (size_t)3 * GC * (a.d.dim16 + 1) * 4;
  const int rc = lds_attr((const void*)gla_read_kernel<T, NV>, lds);
  if (rc) return rc;
  hipLaunchKernelGGL((gla_read_kernel<T, NV>), dim3(nchunks, a.heads), dim3(256), lds, st, a);
  return VUI_OK;
}

template <typename T>
static int chunk_go(const GlaArgs& a, hipStream_t st) {
  const int nchunks = (a.M + GC - 1) / GC;
  const size_t lds = (size_t)GC * (a.d.dim16 + 1 + a.d.vdim16 + 1) * 4 + (size_t)GC * a.rank * sizeof(T);
  int rc = lds_attr((const void*)gla_chunk_kernel<T>, lds);
  if (rc) return rc;
  hipLaunchKernelGGL(gla_chunk_kernel<T>, dim3(nchunks, a.heads), dim3(256), lds, st, a);
  const int quads = a.heads * a.d.dim16 * a.d.vdim16 / 4;
  hipLaunchKernelGGL(gla_carry_kernel, dim3((quads + 255) / 256), dim3(256), 0, st, a, nchunks);
  const int nt = (a.d.vdim16 / 16 + 1) / 2;
  if (nt <= 1) rc = read_go<T, 1>(a, nchunks, st);
  else if (nt <= 2) rc = read_go<T, 2>(a, nchunks, st);
  else if (nt <= 4) rc = read_go<T, 4>(a, nchunks, st);
  else rc = read_go<T, 8>(a, nchunks, st);
  if (rc) return rc;
  HIP_TRY(hipGetLastError());
  return VUI_OK;
}

int launch_gla_chunk(const GlaArgs& a, hipStream_t st) {
  if (!a.rows.seq || !gla_chunk_ok(a.d) || a.rank > 512) { vui_set_error("gated linear attention by chunks: sizes out of range"); return VUI_EINVAL; }
  return a.dtype == VUI_DTYPE_F32 ? chunk_go<float>(a, st) : chunk_go<bf16_t>(a, st);
}
