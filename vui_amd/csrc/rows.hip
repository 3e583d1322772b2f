// Residual rows of sandwich layers: what a sublayer produced is normed and added, and the next sublayer's input is
// normed, in one pass over the row.  fp32 throughout; a norm divides each of `groups` equal parts of the row by its own
// root mean square.  One workgroup per row, the row in LDS.
#include "common.h"
#include "lm.h"
#include "tile.h"

#define ROWS_THREADS 256

// root mean squares of the parts of `v` (width floats in LDS) -> 1 / rms in inv[g]; every wave takes parts in turn
__device__ __forceinline__ void part_scales(const float* v, float* inv, int width, int groups, float eps) {
  const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, n = width / groups;
  if (groups >= ROWS_THREADS / 64) {
    for (int g = wave; g < groups; g += ROWS_THREADS / 64) {
      float s = 0.f;
      for (int i = lane; i < n; i += 64) { const float a = v[g * n + i]; s = fmaf(a, a, s); }
      s = wave_sum(s);
      if (lane == 0) inv[g] = 1.0f / sqrtf(s / (float)n + eps);
    }
    __syncthreads();
    return;
  }
  // few parts: all waves share each
  __shared__ float red[4][ROWS_THREADS / 64];
  for (int g = 0; g < groups; ++g) {
    float s = 0.f;
    for (int i = threadIdx.x; i < n; i += ROWS_THREADS) { const float a = v[g * n + i]; s = fmaf(a, a, s); }
    s = wave_sum(s);
    if (lane == 0) red[g][wave] = s;
  }
  __syncthreads();
  if ((int)threadIdx.x < groups) {
    const float* r = red[threadIdx.x];
    inv[threadIdx.x] = 1.0f / sqrtf(((r[0] + r[1]) + (r[2] + r[3])) / (float)n + eps);
  }
  __syncthreads();
}

template <typename T>
__global__ __launch_bounds__(ROWS_THREADS) void lm_rows_kernel(const RowArgs p) {
  extern __shared__ __align__(16) float rl[];  // row (w64), 1 / rms (groups)
  float* inv = rl + p.w64;
  const int m = blockIdx.x, tid = threadIdx.x, n = p.width / p.groups;
  float* xr = p.x + (size_t)m * p.w64;
  const size_t row16 = (size_t)m;
  if (p.tokens) {
    int64_t t = p.tokens[m];
    t = t < 0 ? 0 : (t >= p.vocab ? p.vocab - 1 : t);
    for (int k = tid; k < p.w64; k += ROWS_THREADS) {
      const float v = k < p.width ? El<T>::ld((const T*)p.embed + (size_t)t * p.width + k) * p.emb_scale : 0.f;
      rl[k] = v;
      if (p.xcat) El<T>::st((T*)p.xcat + tl_off<T>((int)row16, p.w64 + k, 2 * p.w64), v);
    }
    __syncthreads();
  } else if (p.step) {
    for (int k = tid; k < p.w64; k += ROWS_THREADS) rl[k] = k < p.width ? p.y[(size_t)m * p.ldy + k] + p.step[k] : 0.f;
    __syncthreads();
  } else {
    for (int k = tid; k < p.w64; k += ROWS_THREADS) {
      float v = 0.f;
      if (k < p.width) {
        if (p.share) {
          for (int c = 0; c < p.top; ++c) v = fmaf(p.share[(size_t)m * p.top + c], p.y[((size_t)m * p.top + c) * p.ldy + k], v);
        } else {
          v = p.y[(size_t)m * p.ldy + k];
        }
      }
      rl[k] = v;
    }
    __syncthreads();
    part_scales(rl, inv, p.width, p.groups, p.eps);
    for (int k = tid; k < p.width; k += ROWS_THREADS) rl[k] = xr[k] + rl[k] * inv[k / n] * p.post[k];
    __syncthreads();
  }
  for (int k = tid; k < p.w64; k += ROWS_THREADS) {
    xr[k] = rl[k];
    if (p.layer_out && k < p.width) p.layer_out[(size_t)m * p.width + k] = rl[k];
    if (p.to_cat) El<T>::st((T*)p.xcat + tl_off<T>((int)row16, k, 2 * p.w64), rl[k]);
  }
  if (!p.next) return;
  part_scales(rl, inv, p.width, p.groups, p.eps);
  for (int k = tid; k < p.w64; k += ROWS_THREADS)
    El<T>::st((T*)p.xt + tl_off<T>((int)row16, k, p.w64), k < p.width ? rl[k] * inv[k / n] * p.next[k] : 0.f);
}

int launch_lm_rows(const RowArgs& a, hipStream_t st) {
  if (a.M < 1 || a.groups < 1 || a.width % a.groups || a.w64 < a.width || (a.w64 & 63)) { vui_set_error("lm rows: bad shape M=%d width=%d groups=%d", a.M, a.width, a.groups); return VUI_EINVAL; }
  const size_t lds = ((size_t)a.w64 + a.groups) * 4;
  if (lds > 128 * 1024) { vui_set_error("lm rows: width %d too large", a.width); return VUI_EINVAL; }
  const bool f32 = a.dtype == VUI_DTYPE_F32;
  if (lds > 60 * 1024)
    HIP_TRY(hipFuncSetAttribute(f32 ? (const void*)lm_rows_kernel<float> : (const void*)lm_rows_kernel<bf16_t>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds));
  if (f32) hipLaunchKernelGGL(lm_rows_kernel<float>, dim3(a.M), dim3(ROWS_THREADS), lds, st, a);
  else hipLaunchKernelGGL(lm_rows_kernel<bf16_t>, dim3(a.M), dim3(ROWS_THREADS), lds, st, a);
  HIP_TRY(hipGetLastError());
  return VUI_OK;
}
