// The sampler for vocabularies that do not fit the registers of a workgroup (more than 8192 entries): the same kept
// sets, tie rules and random stream as sample_kernel (sample.h), with the logits re-read from memory in every pass.
//
// One 1024-thread workgroup per row.  Nucleus and top-k cuts are digit searches on order-preserving keys, by mass (in
// integers, so the kept set does not depend on the order of addition) and by count; both end in one rule "every key
// above thr and the first n of those equal to it in index order".  The draw walks 64-entry segments in index order.
#include "common.h"
#include "internal.h"
#include "sample.h"

#define SW_THREADS 1024
#define SW_WAVES (SW_THREADS / WAVE)
#define SW_SEGS 8192  // 64-entry segments: up to 524288 entries

struct WideShared {
  float wseg[SW_SEGS];
  uint16_t tseg[SW_SEGS];
  unsigned long long mass[256], tot[SW_WAVES];
  int hist[256];
  float red[SW_WAVES];
  int ired[SW_WAVES], scan[SW_WAVES];
  float fscan[SW_WAVES];
  int pick, seg;
  float before;
  int digit, over;
};

template <typename T>
__global__ __launch_bounds__(SW_THREADS) void sample_wide_kernel(const SampleArgs p) {
  __shared__ __align__(16) WideShared sh;
  const int b = blockIdx.x, tid = threadIdx.x, wave = __builtin_amdgcn_readfirstlane(tid >> 6), lane = tid & 63;
  const int CS = p.CS;
  const T* lg = (const T*)p.logits + (size_t)b * CS;
  const float temp = p.dev ? p.dev->temperature : p.temperature;
  const int topk = p.dev ? p.dev->top_k : p.top_k;
  const uint64_t seed = p.dev ? p.dev->seed : p.seed;
  const bool greedy = topk == 1 || !(temp > 0.f);
  const float div = greedy ? 1.0f : temp;
  const int sb = p.state_rows ? p.state_rows[b] : b;
  const float* counts = (p.rep_counts && p.penalty > 1.0f) ? p.rep_counts + (size_t)sb * CS : nullptr;
  auto value = [&](int j) { return sample_value(El<T>::ld(lg + j), p.bias, j, counts, p.penalty, div); };

  // maximum, lowest index first
  float m = -INFINITY;
  int mi = 0x7fffffff;
  for (int j = tid; j < CS; j += SW_THREADS) {
    const float v = value(j);
    if (v > m) { m = v; mi = j; }
  }
  {
    const float wm = rows_max(group16_max(m));
    const int cand = wave_min_i(m == wm ? mi : 0x7fffffff);
    if (lane == 0) { sh.red[wave] = wm; sh.ired[wave] = cand; }
  }
  __syncthreads();
  float M = sh.red[0];
  int Mi = sh.ired[0];
  for (int w = 1; w < SW_WAVES; ++w) {
    if (sh.red[w] > M) { M = sh.red[w]; Mi = sh.ired[w]; }
    else if (sh.red[w] == M) Mi = min(Mi, sh.ired[w]);
  }
  if (Mi < 0 || Mi >= CS) Mi = 0;  // no ordinary number among the logits: still an index
  int pick = Mi;
  if (!greedy) {
    uint32_t thr = 0u;                    // kept: key > thr, and the first `ties` keys equal to it
    unsigned long long ties = ~0ull;
    if (p.top_p > 0.f) {
      unsigned long long mine = 0ull;
      auto mass_of = [&](float v) { return (unsigned long long)(__expf(v - M) * 4294967296.0f); };
      for (int j = tid; j < CS; j += SW_THREADS) mine += mass_of(value(j));
#pragma unroll
      for (int off = 32; off >= 1; off >>= 1) mine += shfl_down_u64(mine, off);
      if (lane == 0) sh.tot[wave] = mine;
      __syncthreads();
      unsigned long long Z = 0ull;
      for (int w = 0; w < SW_WAVES; ++w) Z += sh.tot[w];
      unsigned long long rem = (unsigned long long)((double)p.top_p * (double)Z);
      unsigned long long unit = 0ull;  // mass of one key of the boundary class
      for (int shift = 24; shift >= 0; shift -= 8) {
        if (tid < 256) sh.mass[tid] = 0ull;
        __syncthreads();
        for (int j = tid; j < CS; j += SW_THREADS) {
          const float v = value(j);
          const uint32_t k = float_key(v);
          const unsigned long long q = mass_of(v);
          if (q && (shift == 24 || (k >> (shift + 8)) == (thr >> (shift + 8)))) atomicAdd(&sh.mass[(k >> shift) & 255], q);
        }
        __syncthreads();
        // the lowest digit whose mass above still fits the budget
        unsigned long long above = 0ull;
        int digit = 255;
        while (digit > 0 && above + sh.mass[digit] <= rem) above += sh.mass[digit--];
        rem -= above;
        thr |= (uint32_t)digit << shift;
        unit = sh.mass[digit];
        __syncthreads();
      }
      int eq = 0;
      for (int j = tid; j < CS; j += SW_THREADS) eq += float_key(value(j)) == thr;
      eq = wave_sum_i(eq);
      if (lane == 0) sh.ired[wave] = eq;
      __syncthreads();
      int n_eq = 0;
      for (int w = 0; w < SW_WAVES; ++w) n_eq += sh.ired[w];
      __syncthreads();
      unit = n_eq > 0 ? unit / (unsigned long long)n_eq : 0ull;
      ties = unit ? rem / unit + 1ull : ~0ull;
    }
    if (topk > 0 && topk < CS) {
      const uint32_t floor_key = thr;  // everything below is already out
      uint32_t t = 0u;
      int need = topk;
      bool enough = true;
      for (int shift = 24; shift >= 0 && enough; shift -= 8) {
        if (tid < 256) sh.hist[tid] = 0;
        __syncthreads();
        for (int j = tid; j < CS; j += SW_THREADS) {
          const uint32_t k = float_key(value(j));
          if (k >= floor_key && (shift == 24 || (k >> (shift + 8)) == (t >> (shift + 8)))) atomicAdd(&sh.hist[(k >> shift) & 255], 1);
        }
        __syncthreads();
        int digit = 255, over = 0;
        while (digit >= 0 && over + sh.hist[digit] < need) over += sh.hist[digit--];
        if (digit < 0) enough = false;  // the nucleus holds fewer than k
        else { t |= (uint32_t)digit << shift; need -= over; }
        __syncthreads();
      }
      if (enough) {
        const unsigned long long quota = p.exact_k ? (unsigned long long)need : ~0ull;
        if (t > floor_key) ties = quota;
        else ties = quota < ties ? quota : ties;
        thr = t;
      }
    }
    // kept weights and ties per segment of 64 entries, in index order
    const int nseg = (CS + WAVE - 1) / WAVE;
    for (int s = wave; s < nseg; s += SW_WAVES) {
      const int j = s * WAVE + lane;
      float v = 0.f;
      uint32_t k = 0u;
      if (j < CS) { v = value(j); k = float_key(v); }
      const bool above = j < CS && k > thr, eq = j < CS && k == thr;
      const unsigned long long bal = __ballot(eq);
      const float w = wave_sum(above ? __expf(v - M) : 0.f);
      if (lane == 0) { sh.wseg[s] = w; sh.tseg[s] = (uint16_t)__builtin_popcountll(bal); }
    }
    __syncthreads();
    // eight neighbouring segments per thread: ties ahead of them, then their weights with the ties that are kept
    const float wtie = __expf(__uint_as_float((thr & 0x80000000u) ? (thr & 0x7fffffffu) : ~thr) - M);  // weight of a boundary key
    constexpr int SPT = SW_SEGS / SW_THREADS;
    int tl = 0;
#pragma unroll
    for (int i = 0; i < SPT; ++i) { const int s = tid * SPT + i; tl += s < nseg ? sh.tseg[s] : 0; }
    int incl = tl;
#pragma unroll
    for (int off = 1; off < 64; off <<= 1) { const int o = __shfl_up(incl, off); if (lane >= off) incl += o; }
    if (lane == WAVE - 1) sh.scan[wave] = incl;
    __syncthreads();
    int tbefore = incl - tl;
    for (int w = 0; w < wave; ++w) tbefore += sh.scan[w];
    float wl = 0.f;
    {
      int tb = tbefore;
#pragma unroll
      for (int i = 0; i < SPT; ++i) {
        const int s = tid * SPT + i;
        if (s < nseg) {
          const int n = sh.tseg[s];
          const int keep = (unsigned long long)tb >= ties ? 0 : (ties - tb < (unsigned long long)n ? (int)(ties - tb) : n);
          tb += n;
          wl += sh.wseg[s] + (keep > 0 ? (float)keep * wtie : 0.f);  // without a cut thr is no logit
        }
      }
    }
    float winc = wl;
#pragma unroll
    for (int off = 1; off < 64; off <<= 1) { const float o = __shfl_up(winc, off); if (lane >= off) winc += o; }
    if (lane == WAVE - 1) sh.fscan[wave] = winc;
    if (tid == 0) sh.pick = -1;
    __syncthreads();
    float base = 0.f, total = 0.f;
    for (int w = 0; w < SW_WAVES; ++w) { if (w < wave) base += sh.fscan[w]; total += sh.fscan[w]; }
    const uint32_t frame = p.frame_ctr ? (uint32_t)p.frame_ctr[0] : 0u;
    const uint32_t rnd = philox_u32(seed, frame, (uint32_t)sb, (uint32_t)p.codebook, 0u);
    const float target = (float)(rnd >> 8) * (1.0f / 16777216.0f) * total;
    float run = base + winc - wl;
    if (target >= run && target < run + wl) {
      // this thread's segments, then the entries of the one that holds the target
      int tb = tbefore, last = -1;
      bool done = false;
      for (int i = 0; i < SPT && !done; ++i) {
        const int s = tid * SPT + i;
        if (s >= nseg) break;
        for (int j = s * WAVE; j < min((s + 1) * WAVE, CS) && !done; ++j) {
          const float v = value(j);
          const uint32_t k = float_key(v);
          bool keep = k > thr;
          if (k == thr) keep = (unsigned long long)(tb++) < ties;
          if (keep) {
            run += __expf(v - M);
            last = j;
            if (run > target) done = true;
          }
        }
      }
      if (last >= 0) atomicMax(&sh.pick, last);
    }
    __syncthreads();
    if (sh.pick >= 0) pick = sh.pick;
  }
  if (tid == 0) {
    p.out[(size_t)b * p.out_stride + p.out_col] = (int64_t)pick;
    if (counts)
      rep_push(p.rep_counts + (size_t)sb * CS, p.rep_hist ? p.rep_hist + (size_t)sb * p.window : nullptr,
               p.rep_pos ? p.rep_pos + sb * 2 : nullptr, p.window, pick);
  }
}

int launch_sample_wide(const SampleArgs& a, hipStream_t st) {
  if (a.CS < 1 || a.CS > SW_SEGS * WAVE || a.B < 1 || a.tok_out || a.eos_prob || a.pad_to > a.pad_from) {
    vui_set_error("sample: vocabulary of %d entries out of range (max %d)", a.CS, SW_SEGS * WAVE);
    return VUI_EINVAL;
  }
  if (a.dtype == VUI_DTYPE_F32) hipLaunchKernelGGL(sample_wide_kernel<float>, dim3(a.B), dim3(SW_THREADS), 0, st, a);
  else hipLaunchKernelGGL(sample_wide_kernel<bf16_t>, dim3(a.B), dim3(SW_THREADS), 0, st, a);
  HIP_TRY(hipGetLastError());
  return VUI_OK;
}
