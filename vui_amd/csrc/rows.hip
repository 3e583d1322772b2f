// Residual rows of sandwich layers: what a sublayer produced is normed and added, and the next sublayer's input is
// normed, in one pass over the row.  fp32 throughout; a norm divides each of `groups` equal parts of the row by its own
// root mean square.  One workgroup per row, which stays in registers, or in LDS where its parts do not fit the waves.  For
// few rows the router of an expert layer reads the normed row here as well, and a single row is routed.
#include "common.h"
#include "lm.h"
#include "route.h"
#include "tile.h"

// root mean squares of the parts of `v` (width floats in LDS) -> 1 / rms in inv[g].  A team of waves sums a part when
// there are fewer parts than waves; red: max(groups, waves) floats.
template <int NT>
__device__ __forceinline__ void part_scales(const float* v, float* inv, float* red, int width, int groups, float eps) {
  constexpr int WAVES = NT / 64;
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, n = width / groups;
  const int wp = groups < WAVES ? WAVES / groups : 1, teams = WAVES / wp, sub = wave % wp;
  for (int g = wave / wp; g < groups && wave < teams * wp; g += teams) {
    const float* q = v + g * n;
    float s = 0.f;
#pragma unroll 4
    for (int i = sub * 64 + lane; i < n; i += wp * 64) s = fmaf(q[i], q[i], s);
    s = wave_sum(s);
    if (lane == 0) red[g * wp + sub] = s;
  }
  __syncthreads();
  for (int g = threadIdx.x; g < groups; g += NT) {
    float s = 0.f;
    for (int w = 0; w < wp; ++w) s += red[g * wp + w];
    inv[g] = 1.0f / sqrtf(s / (float)n + eps);
  }
  __syncthreads();
}

// router logits of the normed row in LDS: a wave takes blocks of 64 columns, a lane 16 columns of one expert
template <typename T>
__device__ __forceinline__ void route_logits(const RowArgs& p, const float* v, float* red, int m) {
  constexpr int EP = Tl<T>::EP, P = 16 / EP;
  const int NT = blockDim.x, WAVES = NT >> 6;
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, l16 = lane & 15, kg = lane >> 4, nk = p.w64 >> 6;
  for (int b = 0; b < p.experts16 >> 4; ++b) {
    const T* w = (const T*)p.w_router + (size_t)b * nk * 1024 + lane * EP;
    float s = 0.f;
    for (int k = wave; k < nk; k += WAVES) {
      uint4 q[P];
#pragma unroll
      for (int h = 0; h < P; ++h) q[h] = *reinterpret_cast<const uint4*>(w + (size_t)k * 1024 + 64 * EP * h);
      const float* c = v + k * 64 + kg * 16;
#pragma unroll
      for (int h = 0; h < P; ++h) {
        const T* e = reinterpret_cast<const T*>(&q[h]);
#pragma unroll
        for (int i = 0; i < EP; ++i) s = fmaf(El<T>::ld(e + i), c[h * EP + i], s);
      }
    }
    s = rows_sum(s);
    if (kg == 0) red[wave * p.experts16 + b * 16 + l16] = s;
  }
  __syncthreads();
  for (int e = threadIdx.x; e < p.experts16; e += NT) {
    float s = p.router_bias[e];
    for (int w = 0; w < WAVES; ++w) s += red[w * p.experts16 + e];
    p.rlog[(size_t)m * p.experts16 + e] = s;
  }
  if (p.M > 1) return;
  // a single row: the tiles of its experts are its choices as they come
  __threadfence_block();
  __syncthreads();
  if (wave == 0) {
    route_row(p.route, 0);
    __threadfence_block();
    for (int i = lane; i < p.route.top * p.route.tile_rows; i += 64) p.route.ent[i] = i % p.route.tile_rows ? -1 : i / p.route.tile_rows;
    if (lane < p.route.top) p.route.tile_e[lane] = p.route.choice[lane];
    if (lane == 0) p.route.n_tiles[0] = p.route.top;
  }
}

template <typename T, int NT>
__global__ __launch_bounds__(NT) void lm_rows_kernel(const RowArgs p) {
  extern __shared__ __align__(16) float rl[];  // row (w64), 1 / rms (groups), sums
  float *inv = rl + p.w64, *red = inv + p.groups;
  const int m = blockIdx.x, tid = threadIdx.x, n = p.width / p.groups;
  float* xr = p.x + (size_t)m * p.w64;
  const bool add = !p.tokens && !p.step;
  if (p.tokens) {
    int64_t t = p.tokens[m];
    t = t < 0 ? 0 : (t >= p.vocab ? p.vocab - 1 : t);
    for (int k = tid; k < p.w64; k += NT) {
      const float v = k < p.width ? El<T>::ld((const T*)p.embed + (size_t)t * p.width + k) * p.emb_scale : 0.f;
      rl[k] = v;
      if (p.xcat) El<T>::st((T*)p.xcat + tl_off<T>(m, p.w64 + k, 2 * p.w64), v);
    }
    __syncthreads();
  }
  float4 old = make_float4(0.f, 0.f, 0.f, 0.f), post = old, next = old;  // of the thread's first quad, requested ahead of use
  const int k1 = min(tid * 4, p.w64 - 4);
  if (add) {
    old = *reinterpret_cast<const float4*>(xr + k1);
    post = *reinterpret_cast<const float4*>(p.post + k1);
  }
  if (p.next) next = *reinterpret_cast<const float4*>(p.next + k1);
  if (!p.tokens) {
    for (int k = tid * 4; k < p.w64; k += NT * 4) {
      tl_f32x4 v = {0.f, 0.f, 0.f, 0.f};
      if (k < p.ldy) {  // what is behind the width is zero
        if (add && p.share) {
          const float *y = p.y + (size_t)m * p.top * p.ldy + k, *s = p.share + (size_t)m * p.top;
#pragma unroll 4
          for (int c = 0; c < p.top; ++c) v += s[c] * *reinterpret_cast<const tl_f32x4*>(y + (size_t)c * p.ldy);
        } else {
          v = *reinterpret_cast<const tl_f32x4*>(p.y + (size_t)m * p.ldy + k);
        }
      }
      if (p.step) v += *reinterpret_cast<const tl_f32x4*>(p.step + k);
      *reinterpret_cast<tl_f32x4*>(rl + k) = v;
    }
    __syncthreads();
  }
  if (add) part_scales<NT>(rl, inv, red, p.width, p.groups, p.eps);
  for (int k = tid * 4; k < p.w64; k += NT * 4) {
    tl_f32x4 v = *reinterpret_cast<const tl_f32x4*>(rl + k);
    if (add) {
      if (k != k1) {
        old = *reinterpret_cast<const float4*>(xr + k);
        post = *reinterpret_cast<const float4*>(p.post + k);
      }
      const float o[4] = {old.x, old.y, old.z, old.w}, w[4] = {post.x, post.y, post.z, post.w};
#pragma unroll
      for (int i = 0; i < 4; ++i) v[i] = k + i < p.width ? o[i] + v[i] * inv[(k + i) / n] * w[i] : 0.f;
      *reinterpret_cast<tl_f32x4*>(rl + k) = v;
    }
    *reinterpret_cast<tl_f32x4*>(xr + k) = v;
    const float f[4] = {v[0], v[1], v[2], v[3]};
    if (p.to_cat) Tl<T>::st4((T*)p.xcat + tl_off<T>(m, k, 2 * p.w64), f);
    if (p.layer_out)
      for (int i = 0; i < 4; ++i) if (k + i < p.width) p.layer_out[(size_t)m * p.width + k + i] = f[i];
  }
  if (!p.next) return;
  __syncthreads();
  part_scales<NT>(rl, inv, red, p.width, p.groups, p.eps);
  for (int k = tid * 4; k < p.w64; k += NT * 4) {
    if (k != k1) next = *reinterpret_cast<const float4*>(p.next + k);
    const float w[4] = {next.x, next.y, next.z, next.w};
    float f[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) f[i] = k + i < p.width ? rl[k + i] * inv[(k + i) / n] * w[i] : 0.f;
    T* dst = (T*)p.xt + tl_off<T>(m, k, p.w64);
    Tl<T>::st4(dst, f);
    if (p.rlog) {  // the router reads what the product of more rows would: the rounded row
      T r[4];
#pragma unroll
      for (int i = 0; i < 4; ++i) { El<T>::st(&r[i], f[i]); f[i] = El<T>::ld(&r[i]); }
      *reinterpret_cast<float4*>(rl + k) = make_float4(f[0], f[1], f[2], f[3]);
    }
  }
  if (!p.rlog) return;
  __syncthreads();
  route_logits<T>(p, rl, red, m);
}

// The same where a wave's lanes hold four columns each of one part (parts of whole quads, no more than 16 waves for all of
// them): the row stays in registers, and a part of up to 256 columns needs no barrier.
template <typename T>
__global__ __launch_bounds__(1024) void lm_rows_quad_kernel(const RowArgs p, int wp) {
  extern __shared__ __align__(16) float rl[];  // for the router: row (w64), sums
  __shared__ float red[2][16];
  const int m = blockIdx.x, tid = threadIdx.x, wave = __builtin_amdgcn_readfirstlane(tid >> 6), lane = tid & 63, n = p.width / p.groups;
  const int g = wave / wp, at = ((wave - g * wp) * 64 + lane) * 4;
  const bool live = at < n, add = !p.tokens && !p.step;
  const int k = g * n + min(at, n - 4);
  auto part_scale = [&](const tl_f32x4& v, int which) {
    float s = live ? (v[0] * v[0] + v[1] * v[1]) + (v[2] * v[2] + v[3] * v[3]) : 0.f;
    s = wave_sum(s);
    if (wp > 1) {
      if (lane == 0) red[which][wave] = s;
      __syncthreads();
      s = 0.f;
      for (int w = 0; w < wp; ++w) s += red[which][g * wp + w];
    }
    return 1.0f / sqrtf(s / (float)n + p.eps);
  };
  float* xr = p.x + (size_t)m * p.w64;
  tl_f32x4 v, old, post, next;
  if (add) {
    old = *reinterpret_cast<const tl_f32x4*>(xr + k);
    post = *reinterpret_cast<const tl_f32x4*>(p.post + k);
  } else if (p.step) {
    old = *reinterpret_cast<const tl_f32x4*>(p.step + k);
  }
  if (p.next) next = *reinterpret_cast<const tl_f32x4*>(p.next + k);
  if (p.tokens) {
    int64_t t = p.tokens[m];
    t = t < 0 ? 0 : (t >= p.vocab ? p.vocab - 1 : t);
    const T* e = (const T*)p.embed + (size_t)t * p.width + k;
    const float f[4] = {El<T>::ld(e) * p.emb_scale, El<T>::ld(e + 1) * p.emb_scale, El<T>::ld(e + 2) * p.emb_scale, El<T>::ld(e + 3) * p.emb_scale};
    v = tl_f32x4{f[0], f[1], f[2], f[3]};
    if (p.xcat && live) Tl<T>::st4((T*)p.xcat + tl_off<T>(m, p.w64 + k, 2 * p.w64), f);
  } else if (add && p.share) {
    const float *y = p.y + (size_t)m * p.top * p.ldy + k, *s = p.share + (size_t)m * p.top;
    v = tl_f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll 4
    for (int c = 0; c < p.top; ++c) v += s[c] * *reinterpret_cast<const tl_f32x4*>(y + (size_t)c * p.ldy);
  } else {
    v = *reinterpret_cast<const tl_f32x4*>(p.y + (size_t)m * p.ldy + k);
    if (p.step) v += old;
  }
  if (add) {
    const float r = part_scale(v, 0);
    v = old + v * r * post;
  }
  const float f[4] = {v[0], v[1], v[2], v[3]}, none[4] = {0.f, 0.f, 0.f, 0.f};
  if (live) {
    *reinterpret_cast<tl_f32x4*>(xr + k) = v;
    if (p.to_cat) Tl<T>::st4((T*)p.xcat + tl_off<T>(m, k, 2 * p.w64), f);
    if (p.layer_out)
      for (int i = 0; i < 4; ++i) p.layer_out[(size_t)m * p.width + k + i] = f[i];
  }
  const int pad = p.width + 4 * tid;  // columns behind the width
  if (pad < p.w64) {
    if (p.xcat && p.tokens) Tl<T>::st4((T*)p.xcat + tl_off<T>(m, p.w64 + pad, 2 * p.w64), none);
    if (p.to_cat) Tl<T>::st4((T*)p.xcat + tl_off<T>(m, pad, 2 * p.w64), none);
    if (p.next) Tl<T>::st4((T*)p.xt + tl_off<T>(m, pad, p.w64), none);
    if (p.rlog) *reinterpret_cast<tl_f32x4*>(rl + pad) = tl_f32x4{0.f, 0.f, 0.f, 0.f};
  }
  if (!p.next) return;
  v = v * part_scale(v, 1) * next;
  float o[4] = {v[0], v[1], v[2], v[3]};
  if (live) Tl<T>::st4((T*)p.xt + tl_off<T>(m, k, p.w64), o);
  if (!p.rlog) return;
  T r[4];  // the router reads what the product of more rows would: the rounded row
#pragma unroll
  for (int i = 0; i < 4; ++i) { El<T>::st(&r[i], o[i]); o[i] = El<T>::ld(&r[i]); }
  if (live) *reinterpret_cast<float4*>(rl + k) = make_float4(o[0], o[1], o[2], o[3]);
  __syncthreads();
  route_logits<T>(p, rl, rl + p.w64, m);
}

template <typename T>
static int quad_go(const RowArgs& a, int wp, hipStream_t st) {
  const int waves = a.groups * wp;
  const size_t lds = a.rlog ? ((size_t)a.w64 + waves * a.experts16) * 4 : 0;
  if (lds > 60 * 1024) HIP_TRY(hipFuncSetAttribute((const void*)lm_rows_quad_kernel<T>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds));
  hipLaunchKernelGGL(lm_rows_quad_kernel<T>, dim3(a.M), dim3(64 * waves), lds, st, a, wp);
  HIP_TRY(hipGetLastError());
  return VUI_OK;
}

bool lm_rows_routes(int M, int experts16) { return M <= 16 && experts16 <= 128; }

template <typename T, int NT>
static int rows_go(const RowArgs& a, hipStream_t st) {
  const int teams = a.groups < NT / 64 ? NT / 64 : a.groups, sums = a.rlog ? NT / 64 * a.experts16 : 0;
  const size_t lds = ((size_t)a.w64 + a.groups + (sums > teams ? sums : teams)) * 4;
  if (lds > 128 * 1024) { vui_set_error("lm rows: width %d too large", a.width); return VUI_EINVAL; }
  if (lds > 60 * 1024) HIP_TRY(hipFuncSetAttribute((const void*)lm_rows_kernel<T, NT>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds));
  hipLaunchKernelGGL((lm_rows_kernel<T, NT>), dim3(a.M), dim3(NT), lds, st, a);
  HIP_TRY(hipGetLastError());
  return VUI_OK;
}

int launch_lm_rows(const RowArgs& a, hipStream_t st) {
  if (a.M < 1 || a.groups < 1 || a.width % a.groups || a.w64 < a.width || (a.w64 & 63) || (a.ldy & 3) || (a.rlog && !lm_rows_routes(a.M, a.experts16))) {
    vui_set_error("lm rows: bad shape M=%d width=%d groups=%d", a.M, a.width, a.groups);
    return VUI_EINVAL;
  }
  const int n = a.width / a.groups, wp = (n + 255) / 256;
  if (n % 4 == 0 && a.groups * wp <= 16) return a.dtype == VUI_DTYPE_F32 ? quad_go<float>(a, wp, st) : quad_go<bf16_t>(a, wp, st);
  if (a.M <= 64) return a.dtype == VUI_DTYPE_F32 ? rows_go<float, 1024>(a, st) : rows_go<bf16_t, 1024>(a, st);
  return a.dtype == VUI_DTYPE_F32 ? rows_go<float, 256>(a, st) : rows_go<bf16_t, 256>(a, st);
}
