// The choice of experts of one row, shared by the routing launches and the row kernel.
#pragma once
#include "lm.h"

// one wave; picks in order of falling logits, so "behind the last pick" needs no list of what was taken
__device__ __forceinline__ void route_row(const RouteArgs& p, int m) {
  const int lane = threadIdx.x & 63;
  const float* z = p.logits + (size_t)m * p.ldl;
  float last = INFINITY, vmax = 0.f, sum = 0.f, mine = 0.f;
  int last_e = -1;
  for (int c = 0; c < p.top; ++c) {
    float bv = -INFINITY;
    int be = 0x7fffffff;
    for (int e = lane; e < p.E; e += 64) {
      const float v = z[e];
      if ((v < last || (v == last && e > last_e)) && (v > bv || be == 0x7fffffff)) { bv = v; be = e; }
    }
#pragma unroll
    for (int o = 32; o >= 1; o >>= 1) {
      const float ov = __shfl_xor(bv, o);
      const int oe = __shfl_xor(be, o);
      if (oe != 0x7fffffff && (be == 0x7fffffff || ov > bv || (ov == bv && oe < be))) { bv = ov; be = oe; }
    }
    if (c == 0) vmax = bv;
    const float w = expf(bv - vmax);
    sum += w;
    if (lane == c) mine = w;
    if (lane == 0) p.choice[(size_t)m * p.top + c] = be < p.E ? be : 0;
    last = bv;
    last_e = be;
  }
  if (lane < p.top) p.share[(size_t)m * p.top + lane] = mine / sum;
}
