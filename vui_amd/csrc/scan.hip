// Gated recurrence S_t = a_t S_(t-1) + b_t over the positions of one sequence, channel by channel, fp32 throughout;
// output S_t * gate_t in the tiled operand layout.  (a, b) pairs come from the projection's epilogue.
//
// The positions are cut into chunks of 32: one launch folds every chunk to its (product of a, end value from zero),
// the second starts each chunk from the fold of the chunks before it.  The incoming state is copied next to the folds
// first, because the last chunk's workgroup overwrites it while others still start from it.
#include "common.h"
#include "lm.h"
#include "tile.h"

__global__ __launch_bounds__(256) void scan_fold_kernel(const ScanArgs p, int nchunks) {
  const int ch = blockIdx.x * 256 + threadIdx.x, c = blockIdx.y;
  if (ch >= p.W) return;
  if (c == nchunks) {  // the state the sequence starts from
    p.agg[(size_t)nchunks * p.ld + ch] = make_float2(0.f, p.from_zero ? 0.f : p.state[ch]);
    return;
  }
  const int t0 = c * LM_SCAN_CHUNK;
  float2 u[LM_SCAN_CHUNK];  // the whole chunk is requested at once
#pragma unroll
  for (int i = 0; i < LM_SCAN_CHUNK; ++i) u[i] = p.upd[(size_t)min(t0 + i, p.T - 1) * p.ld + ch];
  float a = 1.f, b = 0.f;
#pragma unroll
  for (int i = 0; i < LM_SCAN_CHUNK; ++i)
    if (t0 + i < p.T) {
      b = fmaf(u[i].x, b, u[i].y);
      a *= u[i].x;
    }
  p.agg[(size_t)c * p.ld + ch] = make_float2(a, b);
}

template <typename T>
__global__ __launch_bounds__(256) void scan_apply_kernel(const ScanArgs p, int nchunks) {
  const int ch = blockIdx.x * 256 + threadIdx.x, c = blockIdx.y;
  if (ch >= p.W) return;
  const int t0 = c * LM_SCAN_CHUNK;
  float2 u[LM_SCAN_CHUNK];
  T g[LM_SCAN_CHUNK];
#pragma unroll
  for (int i = 0; i < LM_SCAN_CHUNK; ++i) {
    const size_t o = (size_t)min(t0 + i, p.T - 1) * p.ld + ch;
    u[i] = p.upd[o];
    g[i] = ((const T*)p.gate)[o];
  }
  float s;
  if (nchunks == 1) {
    s = p.from_zero ? 0.f : p.state[ch];
  } else {
    s = p.agg[(size_t)nchunks * p.ld + ch].y;
#pragma unroll 8
    for (int k = 0; k < c; ++k) {
      const float2 f = p.agg[(size_t)k * p.ld + ch];
      s = fmaf(f.x, s, f.y);
    }
  }
#pragma unroll
  for (int i = 0; i < LM_SCAN_CHUNK; ++i)
    if (t0 + i < p.T) {
      s = fmaf(u[i].x, s, u[i].y);
      El<T>::st((T*)p.act + tl_off<T>(t0 + i, ch, p.out_k), s * El<T>::ld(&g[i]));
    }
  if (c == nchunks - 1) p.state[ch] = s;
}

int launch_gated_scan(const ScanArgs& a, hipStream_t st) {
  if (a.T < 1 || a.W < 1 || a.ld < a.W) { vui_set_error("gated scan: bad shape T=%d W=%d", a.T, a.W); return VUI_EINVAL; }
  const int nchunks = (a.T + LM_SCAN_CHUNK - 1) / LM_SCAN_CHUNK;
  const int gx = (a.W + 255) / 256;
  if (nchunks > 1) hipLaunchKernelGGL(scan_fold_kernel, dim3(gx, nchunks + 1), dim3(256), 0, st, a, nchunks);
  if (a.dtype == VUI_DTYPE_F32) hipLaunchKernelGGL(scan_apply_kernel<float>, dim3(gx, nchunks), dim3(256), 0, st, a, nchunks);
  else hipLaunchKernelGGL(scan_apply_kernel<bf16_t>, dim3(gx, nchunks), dim3(256), 0, st, a, nchunks);
  HIP_TRY(hipGetLastError());
  return VUI_OK;
}
