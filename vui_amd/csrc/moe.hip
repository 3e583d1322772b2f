// Expert routing: the `top` largest router logits of a row (the lower index wins a tie), shares by softmax over those, and
// the (row, choice) entries sorted by expert, every expert's padded to whole tiles of the products that follow.
#include "common.h"
#include "lm.h"
#include "route.h"
#include "tile.h"

__global__ __launch_bounds__(256) void moe_top_kernel(const RouteArgs p) {
  const int m = blockIdx.x * 4 + (threadIdx.x >> 6);
  if (m < p.M) route_row(p, m);
}

// One workgroup sorts all entries.  Where an entry lands inside its expert's run has no effect on its numbers.
template <bool TOP>
__global__ __launch_bounds__(1024) void moe_sort_kernel(const RouteArgs p) {
  __shared__ int cnt[VUI_LM_MAX_EXPERTS], start[VUI_LM_MAX_EXPERTS], wsum[16];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, n = p.M * p.top;
  cnt[tid] = 0;
  if (TOP) {
    for (int m = wave; m < p.M; m += 16) route_row(p, m);
    __threadfence_block();
  }
  __syncthreads();
  for (int i = tid; i < n; i += 1024) atomicAdd(&cnt[p.choice[i]], 1);
  __syncthreads();
  const int tiles = tid < p.E ? (cnt[tid] + p.tile_rows - 1) / p.tile_rows : 0;
  int s = tiles;  // inclusive sum over the wave
#pragma unroll
  for (int o = 1; o < 64; o <<= 1) {
    const int v = __shfl_up(s, o);
    if (lane >= o) s += v;
  }
  if (lane == 63) wsum[wave] = s;
  __syncthreads();
  for (int w = 0; w < wave; ++w) s += wsum[w];
  const int first = s - tiles;
  for (int t = first; t < s; ++t) p.tile_e[t] = tid;
  for (int i = first * p.tile_rows + (tid < p.E ? cnt[tid] : 0); i < s * p.tile_rows; ++i) p.ent[i] = -1;
  start[tid] = first * p.tile_rows;
  if (tid == 1023) p.n_tiles[0] = s;
  __syncthreads();
  cnt[tid] = 0;
  __syncthreads();
  for (int i = tid; i < n; i += 1024) {
    const int e = p.choice[i];
    p.ent[start[e] + atomicAdd(&cnt[e], 1)] = i;
  }
}

int launch_moe_route(const RouteArgs& a, hipStream_t st) {
  if (a.M < 1 || a.E < 1 || a.E > VUI_LM_MAX_EXPERTS || a.top < 1 || a.top > VUI_LM_MAX_TOP || a.top > a.E || a.ldl < a.E) {
    vui_set_error("expert routing: bad shape M=%d experts=%d top=%d", a.M, a.E, a.top);
    return VUI_EINVAL;
  }
  if (a.M <= 16) {
    hipLaunchKernelGGL(moe_sort_kernel<true>, dim3(1), dim3(1024), 0, st, a);
  } else {
    hipLaunchKernelGGL(moe_top_kernel, dim3((a.M + 3) / 4), dim3(256), 0, st, a);
    hipLaunchKernelGGL(moe_sort_kernel<false>, dim3(1), dim3(1024), 0, st, a);
  }
  HIP_TRY(hipGetLastError());
  return VUI_OK;
}

// one workgroup per 16 entries and slice of the columns; a thread copies pieces of 16 bytes
template <typename T>
__global__ __launch_bounds__(256) void moe_gather_kernel(const RouteArgs p, const T* x, T* out, int nk) {
  constexpr int EP = Tl<T>::EP, P = 16 / EP;
  const int b = blockIdx.x, tid = threadIdx.x, lane = tid & 63;
  if (b * 16 >= p.n_tiles[0] * p.tile_rows) return;
  const int r = min(max(p.ent[b * 16 + (lane & 15)], 0) / p.top, p.M - 1);  // padding entries read row 0
  const T* src = x + (size_t)(r >> 4) * nk * 1024 + ((r & 15) + 16 * (lane >> 4)) * EP;
  T* dst = out + (size_t)b * nk * 1024 + lane * EP;
  for (int i = blockIdx.y * 4 + (tid >> 6); i < nk * P; i += 4 * gridDim.y)
    *reinterpret_cast<uint4*>(dst + (size_t)i * 64 * EP) = *reinterpret_cast<const uint4*>(src + (size_t)i * 64 * EP);
}

int launch_moe_gather(int dtype, const RouteArgs& a, const void* x, void* out, int cols, int max_tiles, hipStream_t st) {
  if (cols < 64 || (cols & 63) || max_tiles < 1 || (a.tile_rows & 15)) { vui_set_error("expert gather: bad shape"); return VUI_EINVAL; }
  const dim3 grid(max_tiles * (a.tile_rows / 16), 2);
  if (dtype == VUI_DTYPE_F32) hipLaunchKernelGGL(moe_gather_kernel<float>, grid, dim3(256), 0, st, a, (const float*)x, (float*)out, cols >> 6);
  else hipLaunchKernelGGL(moe_gather_kernel<bf16_t>, grid, dim3(256), 0, st, a, (const bf16_t*)x, (bf16_t*)out, cols >> 6);
  HIP_TRY(hipGetLastError());
  return VUI_OK;
}
