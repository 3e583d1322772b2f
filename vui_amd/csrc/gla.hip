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

// log of the decay behind its gate's logit: -softplus(-z) / tau
__device__ __forceinline__ float gla_log_sigmoid(const GlaArgs& p, float z) { return -(fmaxf(-z, 0.f) + log1pf(expf(-fabsf(z)))) * p.inv_tau; }

template <typename T> __device__ __forceinline__ void ld4(const T* q, float* o);
template <> __device__ __forceinline__ void ld4<float>(const float* q, float* o) {
  const float4 v = *reinterpret_cast<const float4*>(q);
  o[0] = v.x; o[1] = v.y; o[2] = v.z; o[3] = v.w;
}
template <> __device__ __forceinline__ void ld4<bf16_t>(const bf16_t* q, float* o) {
  const uint2 v = *reinterpret_cast<const uint2*>(q);
  o[0] = bf_lo(v.x); o[1] = bf_hi(v.x); o[2] = bf_lo(v.y); o[3] = bf_hi(v.y);
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
    for (int d0 = 0; d0 < D; d0 += GLA_THREADS / 4) {  // four lanes share the low-rank sum of a channel
      const int d = min(d0 + (tid >> 2), D - 1);
      const float* w = p.w_a2 + ((size_t)h * D + d) * p.rank;
      float z = 0.f;
#pragma unroll 4
      for (int r = tid & 3; r < p.rank; r += 4) z = fmaf(w[r], El<T>::ld(row + c.a + r), z);
      z += dpp_f<DPP_QUAD_XOR1>(z);
      z += dpp_f<DPP_QUAD_XOR2>(z);
      if ((tid & 3) == 0) la[d] = expf(gla_log_sigmoid(p, z + p.a2_bias[h * D + d]));
    }
    for (int d = tid; d < D; d += GLA_THREADS) {
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
#define GLA_SEG 8  // positions a thread sums in a row
template <typename T>
__global__ __launch_bounds__(512) void gla_chunk_kernel(const GlaArgs p) {
  extern __shared__ __align__(16) float gl[];  // sums (GC, D + 1); values (GC, V + 1); low-rank parts (GC, rank4 + 1), then decayed keys (GC, D + 1)
  const int ck = blockIdx.x, h = blockIdx.y, tid = threadIdx.x, lane = tid & 63, l16 = lane & 15, kg = lane >> 4;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int D = p.d.dim16, V = p.d.vdim16, DS = D + 1, VS = V + 1, t0 = ck * GC, n = min(GC, p.M - t0);
  const int R4 = (p.rank + 3) & ~3, RS = R4 + 1;
  float *lb = gl, *lv = gl + GC * DS, *low = lv + GC * VS, *lk = low;
  const GlaCols c = gla_cols(p);
  const T* raw = (const T*)p.raw + (size_t)t0 * p.ld;
  for (int i = tid; i < GC * R4; i += 512) {
    const int t = i / R4, r = i - t * R4;
    low[t * RS + r] = t < n && r < p.rank ? El<T>::ld(raw + (size_t)t * p.ld + c.a + r) : 0.f;
  }
  for (int i = tid; i < GC * V / 4; i += 512) {
    const int t = i / (V >> 2), d = (i - t * (V >> 2)) * 4;
    float v[4];
    ld4<T>(raw + (size_t)min(t, n - 1) * p.ld + c.v + h * V + d, v);
#pragma unroll
    for (int e = 0; e < 4; ++e) lv[t * VS + d + e] = t < n ? v[e] : 0.f;
  }
  __syncthreads();
  for (int i = wave; i < 2 * (D >> 4); i += 8) {  // 16 channels x 16 positions of the gate's logits
    const int d0 = (i >> 1) * 16, t = (i & 1) * 16 + l16;
    const float* w = p.w_a2 + ((size_t)h * D + d0 + l16) * p.rank;
    tl_f32x4 z = {0.f, 0.f, 0.f, 0.f};
    for (int r0 = 0; r0 < R4; r0 += 4) {
      const int r = r0 + kg;
      z = __builtin_amdgcn_mfma_f32_16x16x4f32(r < p.rank ? w[min(r, p.rank - 1)] : 0.f, low[t * RS + r], z, 0, 0, 0);
    }
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const int d = d0 + 4 * kg + e;
      lb[t * DS + d] = t < n ? gla_log_sigmoid(p, z[e] + p.a2_bias[h * D + d]) : 0.f;
    }
  }
  __syncthreads();
  for (int i = tid; i < D * (GC / GLA_SEG); i += 512) {
    const int s = i / D, d = i - s * D;
    float b = 0.f;
#pragma unroll
    for (int t = 0; t < GLA_SEG; ++t) {
      b += lb[(s * GLA_SEG + t) * DS + d];
      lb[(s * GLA_SEG + t) * DS + d] = b;
    }
  }
  __syncthreads();
  for (int i = tid; i < D * (GC / GLA_SEG); i += 512) {
    const int s = i / D, d = i - s * D;
    float k[GLA_SEG], before = 0.f, end = 0.f;
#pragma unroll
    for (int t = 0; t < GLA_SEG; ++t) k[t] = El<T>::ld(raw + (size_t)min(s * GLA_SEG + t, n - 1) * p.ld + c.k + h * D + d);
#pragma unroll
    for (int u = 0; u < GC / GLA_SEG; ++u) {
      if (u == s) before = end;
      end += lb[(u * GLA_SEG + GLA_SEG - 1) * DS + d];
    }
#pragma unroll
    for (int u = 0; u < GLA_SEG; ++u) {
      const int t = s * GLA_SEG + u;
      const float b = before + lb[t * DS + d];
      if (t < n) p.bsum[((size_t)(t0 + t) * p.heads + h) * D + d] = b;
      lk[t * DS + d] = t < n ? k[u] * expf(fminf(end - b, 0.f)) : 0.f;  // positions beyond the portion add nothing
    }
    if (s == 0) p.dec[((size_t)ck * p.heads + h) * D + d] = expf(end);
  }
  __syncthreads();
  float* U = p.upd + ((size_t)ck * p.heads + h) * D * V;
  for (int vt = wave; vt < (V >> 4); vt += 8) {
    float v[GC / 4];
#pragma unroll
    for (int s = 0; s < GC / 4; ++s) v[s] = lv[(4 * s + kg) * VS + vt * 16 + l16];
    for (int d0 = 0; d0 < D; d0 += 16) {
      tl_f32x4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int s = 0; s < GC / 4; ++s) acc = __builtin_amdgcn_mfma_f32_16x16x4f32(v[s], lk[(4 * s + kg) * DS + d0 + l16], acc, 0, 0, 0);
      *reinterpret_cast<tl_f32x4*>(U + (size_t)(d0 + l16) * V + vt * 16 + 4 * kg) = acc;
    }
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

// ---- read: outputs of a chunk; a wave owns the value tiles wave, wave + 8, ... (NV of them) of all positions ----
template <typename T, int NV>
__global__ __launch_bounds__(512) void gla_read_kernel(const GlaArgs p) {
  extern __shared__ __align__(16) float gl[];  // b, q, k (GC, D + 4)
  __shared__ float A[GC][GC + 1], half[8][16][17], red[8][GC];
  const int ck = blockIdx.x, h = blockIdx.y, tid = threadIdx.x, lane = tid & 63, l16 = lane & 15, kg = lane >> 4;
  const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
  const int D = p.d.dim16, V = p.d.vdim16, DS = D + 4, t0 = ck * GC, n = min(GC, p.M - t0), nv = V >> 4;
  float *lb = gl, *lq = gl + GC * DS, *lk = gl + 2 * GC * DS;
  const GlaCols c = gla_cols(p);
  const T* raw = (const T*)p.raw + (size_t)t0 * p.ld;
  for (int i = tid; i < GC * D / 4; i += 512) {
    const int t = i / (D >> 2), d = (i - t * (D >> 2)) * 4, at = min(t, n - 1);
    float b[4], q[4], k[4];
    ld4<float>(p.bsum + ((size_t)(t0 + at) * p.heads + h) * D + d, b);
    ld4<T>(raw + (size_t)at * p.ld + h * D + d, q);
    ld4<T>(raw + (size_t)at * p.ld + c.k + h * D + d, k);
    const float f = t < n ? p.q_scale : 0.f;
    *reinterpret_cast<float4*>(lb + t * DS + d) = t < n ? make_float4(b[0], b[1], b[2], b[3]) : make_float4(0.f, 0.f, 0.f, 0.f);
    *reinterpret_cast<float4*>(lq + t * DS + d) = make_float4(q[0] * f, q[1] * f, q[2] * f, q[3] * f);
    *reinterpret_cast<float4*>(lk + t * DS + d) = t < n ? make_float4(k[0], k[1], k[2], k[3]) : make_float4(0.f, 0.f, 0.f, 0.f);
  }
  // the incoming state comes 16 rows at a time, two loads ahead of their products; the values right away
  const float* S = p.upd + ((size_t)ck * p.heads + h) * D * V + l16;
  int vt[NV];
#pragma unroll
  for (int i = 0; i < NV; ++i) vt[i] = min(wave + 8 * i, nv - 1) * 16;
  float s0[4][NV], s1[4][NV], vv[GC / 4][NV];
  auto fetch = [&](float (*s)[NV], int d0) {
#pragma unroll
    for (int u = 0; u < 4; ++u)
#pragma unroll
      for (int i = 0; i < NV; ++i) s[u][i] = S[(size_t)(min(d0, D - 16) + 4 * u + kg) * V + vt[i]];
  };
  fetch(s0, 0);
  fetch(s1, 16);
#pragma unroll
  for (int u = 0; u < GC / 4; ++u)
#pragma unroll
    for (int i = 0; i < NV; ++i) vv[u][i] = El<T>::ld(raw + (size_t)min(4 * u + kg, n - 1) * p.ld + c.v + h * V + vt[i] + l16);
  __syncthreads();
  {  // the two triangles of 16 positions
    const int o = (tid >> 8) * 16, s = o + (tid & 15), t = o + ((tid >> 4) & 15);
    float a = 0.f;
    if (s <= t && t < n) {
      const float *q = lq + t * DS, *bt = lb + t * DS, *k = lk + s * DS, *bs = lb + s * DS;
#pragma unroll 2
      for (int d = 0; d < D; d += 4) {
        const tl_f32x4 x = *reinterpret_cast<const tl_f32x4*>(q + d) * *reinterpret_cast<const tl_f32x4*>(k + d);
        const tl_f32x4 e = *reinterpret_cast<const tl_f32x4*>(bt + d) - *reinterpret_cast<const tl_f32x4*>(bs + d);
#pragma unroll
        for (int r = 0; r < 4; ++r) a = fmaf(x[r], sizeof(T) == 4 ? expf(e[r]) : __expf(e[r]), a);
      }
    }
    A[t][s] = a;
  }
  {  // later half on earlier half: the waves share the channels
    tl_f32x4 acc = {0.f, 0.f, 0.f, 0.f};
    for (int d0 = wave * 4; d0 < D; d0 += 32) {
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
  if (tid < 256) {
    const int t = tid >> 4, s = tid & 15;
    float a = 0.f;
#pragma unroll
    for (int w = 0; w < 8; ++w) a += half[w][t][s];
    A[16 + t][s] = a;
    A[s][16 + t] = 0.f;
  }
  for (int i = tid; i < GC * D / 4; i += 512) {
    const int t = i / (D >> 2), d = (i - t * (D >> 2)) * 4;
#pragma unroll
    for (int e = 0; e < 4; ++e) lq[t * DS + d + e] *= expf(lb[t * DS + d + e]);
  }
  __syncthreads();
  tl_f32x4 acc[2][NV];
#pragma unroll
  for (int u = 0; u < 2; ++u)
#pragma unroll
    for (int i = 0; i < NV; ++i) acc[u][i] = tl_f32x4{0.f, 0.f, 0.f, 0.f};
  auto state_part = [&](const float (*s)[NV], int d0) {
#pragma unroll
    for (int u = 0; u < 4; ++u) {
      const float qa = lq[l16 * DS + d0 + 4 * u + kg], qb = lq[(16 + l16) * DS + d0 + 4 * u + kg];
#pragma unroll
      for (int i = 0; i < NV; ++i) {
        acc[0][i] = __builtin_amdgcn_mfma_f32_16x16x4f32(s[u][i], qa, acc[0][i], 0, 0, 0);
        acc[1][i] = __builtin_amdgcn_mfma_f32_16x16x4f32(s[u][i], qb, acc[1][i], 0, 0, 0);
      }
    }
  };
  if (ck > 0 || p.rows.pos0 > 0) {
    for (int d0 = 0; d0 < D; d0 += 32) {
      state_part(s0, d0);
      fetch(s0, d0 + 32);
      if (d0 + 16 < D) state_part(s1, d0 + 16);
      fetch(s1, d0 + 48);
    }
  }
  float g[2][NV][4];
#pragma unroll
  for (int u = 0; u < 2; ++u)
#pragma unroll
    for (int i = 0; i < NV; ++i) ld4<T>(raw + (size_t)min(16 * u + l16, n - 1) * p.ld + c.g + h * V + vt[i] + 4 * kg, g[u][i]);
#pragma unroll
  for (int j = 0; j < GC / 4; ++j)
#pragma unroll
    for (int u = 0; u < 2; ++u) {
      const float a = A[16 * u + l16][4 * j + kg];
#pragma unroll
      for (int i = 0; i < NV; ++i) acc[u][i] = __builtin_amdgcn_mfma_f32_16x16x4f32(vv[j][i], a, acc[u][i], 0, 0, 0);
    }
#pragma unroll
  for (int u = 0; u < 2; ++u) {
    float ss = 0.f;
#pragma unroll
    for (int i = 0; i < NV; ++i)
      if (wave + 8 * i < nv)
#pragma unroll
        for (int r = 0; r < 4; ++r) ss = fmaf(acc[u][i][r], acc[u][i][r], ss);
    ss = rows_sum(ss);
    if (kg == 0) red[wave][16 * u + l16] = ss;
  }
  __syncthreads();
#pragma unroll
  for (int u = 0; u < 2; ++u) {
    const int t = 16 * u + l16;
    float ss = 0.f;
#pragma unroll
    for (int w = 0; w < 8; ++w) ss += red[w][t];
    const float r = 1.0f / sqrtf(ss / (float)p.vdim + p.eps);
    if (t >= n) continue;
#pragma unroll
    for (int i = 0; i < NV; ++i) {
      if (wave + 8 * i >= nv) continue;
      const int v0 = vt[i] + 4 * kg;
      float o[4];
#pragma unroll
      for (int e = 0; e < 4; ++e) o[e] = acc[u][i][e] * r * p.head_norm[v0 + e] * silu_exact(g[u][i][e]);
      Tl<T>::st4((T*)p.act + tl_off<T>(t0 + t, h * V + v0, p.d.out_k), o);
    }
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
  const size_t lds = (size_t)3 * GC * (a.d.dim16 + 4) * 4;
  const int rc = lds_attr((const void*)gla_read_kernel<T, NV>, lds);
  if (rc) return rc;
  hipLaunchKernelGGL((gla_read_kernel<T, NV>), dim3(nchunks, a.heads), dim3(512), lds, st, a);
  return VUI_OK;
}

template <typename T>
static int chunk_go(const GlaArgs& a, hipStream_t st) {
  const int nchunks = (a.M + GC - 1) / GC;
  const int low = ((a.rank + 3) & ~3) + 1, keys = a.d.dim16 + 1;
  const size_t lds = (size_t)GC * (keys + a.d.vdim16 + 1 + (low > keys ? low : keys)) * 4;
  int rc = lds_attr((const void*)gla_chunk_kernel<T>, lds);
  if (rc) return rc;
  hipLaunchKernelGGL(gla_chunk_kernel<T>, dim3(nchunks, a.heads), dim3(512), lds, st, a);
  const int quads = a.heads * a.d.dim16 * a.d.vdim16 / 4;
  hipLaunchKernelGGL(gla_carry_kernel, dim3((quads + 255) / 256), dim3(256), 0, st, a, nchunks);
  rc = a.d.vdim16 <= 128 ? read_go<T, 1>(a, nchunks, st) : read_go<T, 2>(a, nchunks, st);
  if (rc) return rc;
  HIP_TRY(hipGetLastError());
  return VUI_OK;
}

int launch_gla_chunk(const GlaArgs& a, hipStream_t st) {
  if (!a.rows.seq || !gla_chunk_ok(a.d) || a.rank > 512) { vui_set_error("gated linear attention by chunks: sizes out of range"); return VUI_EINVAL; }
  return a.dtype == VUI_DTYPE_F32 ? chunk_go<float>(a, st) : chunk_go<bf16_t>(a, st);
}
