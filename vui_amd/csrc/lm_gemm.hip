// The matrix products of the token language models, one kernel template: C (M x N) = X (M x K) W^T (N x K) on the
// matrix cores (bf16 or true fp32), both operands tiled, K split over the waves of a workgroup (partial tiles meet in
// LDS and are added in wave order).  What a layer does with the sums is the epilogue.
//
// Parallel layers: the norm has a single number for its weight, so W norm(x) = s W x with one scale s per row: the product
// runs on the raw residual row and the epilogue scales.  The sum of squares behind s is left by whoever wrote the
// row, in pieces of 16 columns (LM_OUT, the embedding), so no launch is spent on norms.
#include "common.h"
#include "lm.h"
#include "tile.h"

__device__ __forceinline__ float lm_sigmoid(float v) { return 1.0f / (1.0f + expf(-v)); }

// gated feed-forward with clamped branches, two features from interleaved (gate, up) pairs
__device__ __forceinline__ float lm_ff(float g, float u, float limit) {
  g = fminf(g, limit);
  u = fminf(fmaxf(u, -limit), limit);
  return g * lm_sigmoid(1.702f * g) * (u + 1.0f);
}

// rotates two pairs held as (u0, v0, u1, v1); pair indices i, i + 1; pairs at or beyond n pass
__device__ __forceinline__ void lm_rotate2(float* v, const float* rope, int pos, int n, int i) {
#pragma unroll
  for (int k = 0; k < 2; ++k) {
    if (i + k < n) {
      const float2 f = *reinterpret_cast<const float2*>(rope + ((size_t)pos * n + i + k) * 2);
      const float a = v[2 * k], b = v[2 * k + 1];
      v[2 * k] = a * f.x - b * f.y;
      v[2 * k + 1] = b * f.x + a * f.y;
    }
  }
}

// activations of ungated feed-forwards
__device__ __forceinline__ float lm_act(float z, int kind, float pos, float neg) {
  if (kind == VUI_LM_ACT_RELU2) { z = fmaxf(z, 0.f); return z * z; }
  const float m = fminf(z, 0.f);
  return (z > 0.f ? pos * z * z : neg * (expm1f(m) - m)) + 0.5f * z;
}

template <typename T, int MB, int NB, int WAVES, int EPI>
__global__ __launch_bounds__(64 * WAVES) void lm_gemm_kernel(const LmGemm p) {
  constexpr bool SCALED = EPI == LM_IN_ATTN || EPI == LM_IN_GRU_STEP || EPI == LM_IN_GRU_SEQ || EPI == LM_LOGITS;
  constexpr bool GRU = EPI == LM_IN_GRU_STEP || EPI == LM_IN_GRU_SEQ;
  constexpr bool LOGITS = EPI == LM_LOGITS || EPI == LM_HEAD, MOE = EPI == LM_MOE_UP || EPI == LM_MOE_DOWN;
  constexpr bool ROWS_FIRST = EPI == LM_EXPAND_V;  // a lane then holds four consecutive rows of one feature
  constexpr int EP = Tl<T>::EP, P = 16 / EP, TILE = MB * NB * 256;
  __shared__ __align__(16) float part[WAVES * TILE];
  __shared__ float srow[MB * 16];
  const int tid = threadIdx.x, wave = __builtin_amdgcn_readfirstlane(tid >> 6), lane = tid & 63;
  const int l16 = lane & 15, kg = lane >> 4;
  const int MT = MOE ? p.max_tiles : (p.M + 16 * MB - 1) / (16 * MB);
  // tiles of an expert that share features run on one XCD, whose cache then holds those weights: workgroup i is on XCD i % 8
  const int slice = MOE ? (int)blockIdx.x >> 3 : (int)blockIdx.x, t = slice % MT;
  const int m0 = t * 16 * MB, nb0 = (MOE ? (slice / MT) * 8 + ((int)blockIdx.x & 7) : slice / MT) * NB;
  size_t wz = blockIdx.z * p.wz;
  if (MOE) {
    if (t >= p.n_tiles[0] || nb0 >= (p.N >> 4)) return;  // uniform
    wz = (size_t)p.tile_e[t] * p.wz;
  }
  const int nsteps = p.K >> 6;
  const int s0 = nsteps * wave / WAVES, s1 = nsteps * (wave + 1) / WAVES;
  const int MBL = (p.M + 15) >> 4, NBL = p.N >> 4;

  const T* xr[MB];
  const T* wr[NB];
#pragma unroll
  for (int j = 0; j < MB; ++j) {
    if (EPI == LM_MOE_UP && !p.sorted) {
      const int e = p.ent[m0 + 16 * j + l16], r = min(max(e, 0) / p.top, p.x_rows - 1);
      xr[j] = (const T*)p.X + (size_t)(r >> 4) * nsteps * 1024 + ((r & 15) + 16 * kg) * EP;
    } else if (MOE) {
      xr[j] = (const T*)p.X + (size_t)((m0 >> 4) + j) * nsteps * 1024 + lane * EP;
    } else if (LOGITS && p.rowmap) {
      const int r = min(max(p.rowmap[min(m0 + 16 * j + l16, p.M - 1)], 0), p.x_rows - 1);
      xr[j] = (const T*)p.X + (size_t)(r >> 4) * nsteps * 1024 + ((r & 15) + 16 * kg) * EP;
    } else {
      // few rows: lanes without a row re-read the last one instead of fetching a block that is mostly padding
      const int l = MB == 1 && !ROWS_FIRST ? min(l16, p.M - 1 - m0) + 16 * kg : lane;
      xr[j] = (const T*)p.X + (size_t)min((m0 >> 4) + j, MBL - 1) * nsteps * 1024 + l * EP;
    }
  }
#pragma unroll
  for (int i = 0; i < NB; ++i)
    wr[i] = (const T*)p.W + wz + (size_t)min(nb0 + i, NBL - 1) * nsteps * 1024 + lane * EP;

  // What the scale and the epilogue of this wave's first unit will need is requested now, ahead of the operands:
  // fetched where it is used, it would be a chain of dependent loads behind the last product.
  // Scale: TPR neighbouring threads add up one row's sums of squares, in a fixed order.
  constexpr int TPR = WAVES * 64 / (MB * 16) > 64 ? 64 : WAVES * 64 / (MB * 16), NSQ = 4;
  const int sq_r = tid / TPR, sq_q = tid % TPR;
  int sq_m = 0;
  float sq[NSQ], norm = 0.f;
  if (SCALED) {
    sq_m = min(m0 + min(sq_r, MB * 16 - 1), p.M - 1);
    if (LOGITS && p.rowmap) sq_m = min(max(p.rowmap[sq_m], 0), p.x_rows - 1);
#pragma unroll
    for (int i = 0; i < NSQ; ++i) sq[i] = p.ssq[(size_t)sq_m * p.np + min(sq_q + TPR * i, p.np - 1)];
    norm = p.norm[0];
  }
  constexpr bool PRE = MB == 1 && (EPI == LM_IN_ATTN || EPI == LM_IN_GRU_STEP || EPI == LM_OUT);
  const int pm = min(m0 + l16, p.M - 1), pb = min(nb0 + min(wave, NB - 1), NBL - 1);  // row and block of unit `wave`
  int e_slot = 0, e_pos = 0;
  float4 e_a = make_float4(0.f, 0.f, 0.f, 0.f), e_b = e_a, e_c = e_a;
  if (PRE && EPI != LM_OUT) {
    e_slot = lm_slot(p.rows, pm);
    e_pos = lm_pos(p.rows, pm, e_slot);
  }
  if (PRE && EPI == LM_OUT) e_a = *reinterpret_cast<const float4*>(p.x + (size_t)pm * p.d.w64 + pb * 16 + 4 * kg);
  if (PRE && EPI == LM_IN_GRU_STEP && nb0 < p.mix_blocks) {
    const int ch = (nb0 / 3) * 16 + 4 * kg;
    e_a = *reinterpret_cast<const float4*>(p.state + (size_t)e_slot * p.d.gru16 + ch);
    e_b = *reinterpret_cast<const float4*>(p.bz + ch);
    e_c = *reinterpret_cast<const float4*>(p.bx + ch);
  }

  tl_f32x4 acc[NB][MB];
#pragma unroll
  for (int i = 0; i < NB; ++i)
#pragma unroll
    for (int j = 0; j < MB; ++j) acc[i][j] = tl_f32x4{0.f, 0.f, 0.f, 0.f};
  // U steps' loads go out together (a step beyond the wave's last re-reads that one and is not multiplied)
  constexpr int U = WAVES >= 8 && sizeof(T) == 2 ? 4 : 1;
  for (int s = s0; s < s1; s += U) {
    uint4 xa[U][MB][P], wa[U][NB][P];
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const size_t o = (size_t)min(s + u, s1 - 1) * 1024;
#pragma unroll
      for (int h = 0; h < P; ++h) {
#pragma unroll
        for (int i = 0; i < NB; ++i) wa[u][i][h] = *reinterpret_cast<const uint4*>(wr[i] + o + 64 * EP * h);
#pragma unroll
        for (int j = 0; j < MB; ++j) xa[u][j][h] = *reinterpret_cast<const uint4*>(xr[j] + o + 64 * EP * h);
      }
    }
    __builtin_amdgcn_sched_barrier(0);
#pragma unroll
    for (int u = 0; u < U; ++u) {
      if (s + u >= s1) break;  // uniform
#pragma unroll
      for (int h = 0; h < P; ++h)
#pragma unroll
        for (int i = 0; i < NB; ++i)
#pragma unroll
          for (int j = 0; j < MB; ++j)
            acc[i][j] = ROWS_FIRST ? Tl<T>::mma(xa[u][j][h], wa[u][i][h], acc[i][j]) : Tl<T>::mma(wa[u][i][h], xa[u][j][h], acc[i][j]);
    }
  }
#pragma unroll
  for (int i = 0; i < NB; ++i)
#pragma unroll
    for (int j = 0; j < MB; ++j)
      *reinterpret_cast<tl_f32x4*>(&part[wave * TILE + ((i * MB + j) * 64 + lane) * 4]) = acc[i][j];
  if (SCALED) {
    float t = 0.f;
#pragma unroll
    for (int i = 0; i < NSQ; ++i) t += sq_q + TPR * i < p.np ? sq[i] : 0.f;
    for (int i = sq_q + TPR * NSQ; i < p.np; i += TPR) t += p.ssq[(size_t)sq_m * p.np + i];
#pragma unroll
    for (int o = TPR / 2; o >= 1; o >>= 1) t += __shfl_xor(t, o);
    if (sq_r < MB * 16 && sq_q == 0) srow[sq_r] = norm / sqrtf(t / (float)p.width + p.eps);
  }
  __syncthreads();

  const bool mix = GRU && nb0 < p.mix_blocks;  // uniform: a tile is all mixer or all feed-forward (padded that way)
  const int units = mix ? MB : MB * NB;
  for (int u = wave; u < units; u += WAVES) {
    const int j = mix ? u : u % MB, i0 = mix ? 0 : u / MB;
    const int m = m0 + 16 * j + (ROWS_FIRST ? 4 * kg : l16);
    const int nb = nb0 + i0;
    const int n = nb * 16 + (ROWS_FIRST ? l16 : 4 * kg);
    const bool live = (MOE || m < p.M) && nb < NBL;
    const float sc = SCALED ? srow[16 * j + l16] : 1.f;
    float v[4];
    auto gather = [&](int i, float* o) {
      const float* q = part + ((i * MB + j) * 64 + lane) * 4;
      tl_f32x4 a = *reinterpret_cast<const tl_f32x4*>(q);
#pragma unroll
      for (int w = 1; w < WAVES; ++w) a += *reinterpret_cast<const tl_f32x4*>(q + w * TILE);
#pragma unroll
      for (int r = 0; r < 4; ++r) o[r] = a[r] * sc;
    };
    gather(i0, v);

    if (GRU && mix) {
      float xv[4], gv[4];
      gather(NB > 1 ? 1 : 0, xv);
      gather(NB > 2 ? 2 : 0, gv);
      const int ch = (nb / 3) * 16 + 4 * kg;  // blocks come in threes: update gate, candidate, output gate
      if (!live) continue;
      const float4 b0 = PRE ? e_b : *reinterpret_cast<const float4*>(p.bz + ch), b1 = PRE ? e_c : *reinterpret_cast<const float4*>(p.bx + ch);
      const float zb[4] = {b0.x, b0.y, b0.z, b0.w}, xb[4] = {b1.x, b1.y, b1.z, b1.w};
      float keep[4], in[4], sg[4];
#pragma unroll
      for (int r = 0; r < 4; ++r) {
        const float zz = v[r] + zb[r], uu = xv[r] + xb[r];
        const float z = lm_sigmoid(zz);
        keep[r] = lm_sigmoid(-zz);
        in[r] = z * (uu >= 0.f ? uu + 0.5f : lm_sigmoid(uu));
        sg[r] = gv[r] * lm_sigmoid(gv[r]);
      }
      if (EPI == LM_IN_GRU_STEP) {
        float4* sp = reinterpret_cast<float4*>(p.state + (size_t)e_slot * p.d.gru16 + ch);
        const float4 old = e_pos > 0 ? e_a : make_float4(0.f, 0.f, 0.f, 0.f);
        const float4 nw = make_float4(fmaf(keep[0], old.x, in[0]), fmaf(keep[1], old.y, in[1]), fmaf(keep[2], old.z, in[2]),
                                      fmaf(keep[3], old.w, in[3]));
        *sp = nw;
        const float o[4] = {nw.x * sg[0], nw.y * sg[1], nw.z * sg[2], nw.w * sg[3]};
        Tl<T>::st4((T*)p.act + tl_off<T>(m, ch, p.d.out_k), o);
      } else {
        float4* up = reinterpret_cast<float4*>(p.upd + (size_t)m * p.d.gru16 + ch);
        up[0] = make_float4(keep[0], in[0], keep[1], in[1]);
        up[1] = make_float4(keep[2], in[2], keep[3], in[3]);
        Tl<T>::st4((T*)p.sg + (size_t)m * p.d.gru16 + ch, sg);
      }
      continue;
    }
    if (EPI == LM_IN_ATTN || GRU) {
      if (!live) continue;
      if (nb >= p.mix_blocks) {  // (gate, up) pairs
        const int f = (n - p.mix_blocks * 16) >> 1;
        Tl<T>::st2((T*)p.act + tl_off<T>(m, p.d.ff_off + f, p.d.out_k), lm_ff(v[0], v[1], p.limit), lm_ff(v[2], v[3], p.limit));
        continue;
      }
      if (EPI == LM_IN_ATTN) {
        if (nb < p.b_qr) {
          const int dq = p.d.dim16 >> 4, h = nb / dq, o = (nb - h * dq) * 16 + 4 * kg;
          Tl<T>::st4((T*)p.qu + h * p.qu_z + tl_off<T>(m, o, p.d.dim64), v);
        } else if (nb < p.b_c) {
          const int dr = p.d.rot16 >> 4, b = nb - p.b_qr, h = b / dr, o = (b - h * dr) * 16 + 4 * kg;
          const int slot = PRE ? e_slot : lm_slot(p.rows, m), pos = min(max(PRE ? e_pos : lm_pos(p.rows, m, slot), 0), p.rows.S - 1);
          lm_rotate2(v, p.rope, pos, p.rot_pairs, o >> 1);
          Tl<T>::st4((T*)p.qr + h * p.qr_z + tl_off<T, 32>(m, o, p.d.rot32), v);
        } else if (nb < p.b_kr) {
          const int o = (nb - p.b_c) * 16 + 4 * kg;
          *reinterpret_cast<float4*>(p.craw + (size_t)m * p.d.rank16 + o) = make_float4(v[0], v[1], v[2], v[3]);
        } else if (nb < p.b_g) {
          const int o = (nb - p.b_kr) * 16 + 4 * kg;
          const int slot = PRE ? e_slot : lm_slot(p.rows, m), pos = PRE ? e_pos : lm_pos(p.rows, m, slot);
          if (pos >= 0 && pos < p.rows.S) {
            lm_rotate2(v, p.rope, pos, p.rot_pairs, o >> 1);
            Tl<T>::st4((T*)p.kr_cache + (size_t)slot * p.d.s64 * p.d.rot32 + tl_off<T, 32>(pos, o, p.d.rot32), v);
          }
        } else {
          const int o = (nb - p.b_g) * 16 + 4 * kg;
          if (o < p.d.heads16)  // the blocks behind the gates only fill the last tile of the mixer part
            *reinterpret_cast<float4*>(p.gate + (size_t)m * p.d.heads16 + o) =
                make_float4(lm_sigmoid(v[0]), lm_sigmoid(v[1]), lm_sigmoid(v[2]), lm_sigmoid(v[3]));
        }
      }
      continue;
    }
    if (EPI == LM_OUT) {
      float sq = 0.f;
      if (live) {
        float4* xp = reinterpret_cast<float4*>(p.x + (size_t)m * p.d.w64 + n);
        const float4 old = PRE ? e_a : *xp;
        v[0] += old.x; v[1] += old.y; v[2] += old.z; v[3] += old.w;
        *xp = make_float4(v[0], v[1], v[2], v[3]);
        Tl<T>::st4((T*)p.xt + tl_off<T>(m, n, p.d.w64), v);
        sq = (v[0] * v[0] + v[1] * v[1]) + (v[2] * v[2] + v[3] * v[3]);
        if (p.layer_out)
          for (int r = 0; r < 4; ++r) if (n + r < p.width) p.layer_out[(size_t)m * p.width + n + r] = v[r];
      }
      sq = rows_sum(sq);  // the 16 columns of this row's block
      if (live && kg == 0 && nb < p.np) p.ssq_out[(size_t)m * p.np + nb] = sq;
      continue;
    }
    if (LOGITS) {
      if (live)
        for (int r = 0; r < 4; ++r) if (n + r < p.vocab) p.logits[(size_t)m * p.vocab + n + r] = v[r];
      continue;
    }
    if (EPI == LM_PROJ || EPI == LM_PLAIN || EPI == LM_MOE_DOWN) {
      const int r = EPI == LM_MOE_DOWN ? p.ent[m] : m;
      if (!live || r < 0) continue;
      if (EPI != LM_MOE_DOWN && p.bias) {
        const float4 b = *reinterpret_cast<const float4*>(p.bias + n);
        v[0] += b.x; v[1] += b.y; v[2] += b.z; v[3] += b.w;
      }
      if (EPI == LM_PROJ) Tl<T>::st4((T*)p.out + (size_t)r * p.ldo + n, v);
      else Tl<float>::st4((float*)p.out + (size_t)r * p.ldo + n, v);
      continue;
    }
    if (EPI == LM_ACT || EPI == LM_MOE_UP) {
      if (!live) continue;
#pragma unroll
      for (int r = 0; r < 4; ++r) v[r] = lm_act(v[r], p.act_kind, p.act_pos, p.act_neg);
      Tl<T>::st4((T*)p.act + tl_off<T>(m, n, p.act_k), v);
      continue;
    }
    if (EPI == LM_EXPAND_K) {
      if (live) Tl<T>::st4((T*)p.kv_out + blockIdx.z * p.kv_z + tl_off<T>(m, n, p.d.dim64), v);
      continue;
    }
    if (EPI == LM_EXPAND_V) {
      // blocks of 16 value dims x 32 keys; a lane of the attention kernel reads the keys 4 kg .. + 3 of both halves
      if (live) {
        T* dst = (T*)p.kv_out + blockIdx.z * p.kv_z + ((size_t)nb * (p.d.s64 >> 5) + (m >> 5)) * 512 +
                 (l16 + 16 * ((m & 15) >> 2)) * 8 + 4 * ((m & 31) >> 4);
        Tl<T>::st4(dst, v);
      }
      continue;
    }
  }
  if (LOGITS && p.upd_lens && blockIdx.x == 0) {
    if (p.upd_inc) {
      for (int s = tid; s < p.rows.n_slots; s += 64 * WAVES) p.upd_lens[s] += p.upd_inc[s];
    } else {
      for (int b = tid; b < p.upd_rows; b += 64 * WAVES) atomicAdd(&p.upd_lens[lm_slot(p.rows, b)], 1);
    }
  }
}

template <typename T, int MB, int NB, int WAVES, int EPI>
static int go(const LmGemm& g, int nz, hipStream_t st) {
  const bool moe = EPI == LM_MOE_UP || EPI == LM_MOE_DOWN;
  const int nt = (g.N / 16 + NB - 1) / NB;
  const int tiles = moe ? g.max_tiles * ((nt + 7) & ~7) : (g.M + 16 * MB - 1) / (16 * MB) * nt;
  hipLaunchKernelGGL((lm_gemm_kernel<T, MB, NB, WAVES, EPI>), dim3((unsigned)tiles, 1, nz), dim3(64 * WAVES), 0, st, g);
  HIP_TRY(hipGetLastError());
  return VUI_OK;
}

// up to 16 rows: one row block, more waves per tile (the weights are streamed once, latency counts)
template <typename T>
static int pick(int epi, const LmGemm& g, int nz, hipStream_t st) {
  const bool few = g.M <= 16;
  // many rows: tiles of 64 x 64, or 64 x 32 where the former would leave half of the chip idle
  const long tiles = (long)((g.M + 63) / 64) * ((g.N + 63) / 64);
  if (sizeof(T) == 2 && g.M >= 256 && tiles >= 64) {
    const bool wide = tiles >= 160;
    if (epi == LM_PROJ) return wide ? go<T, 4, 4, 4, LM_PROJ>(g, nz, st) : go<T, 4, 2, 4, LM_PROJ>(g, nz, st);
    if (epi == LM_PLAIN) return wide ? go<T, 4, 4, 4, LM_PLAIN>(g, nz, st) : go<T, 4, 2, 4, LM_PLAIN>(g, nz, st);
    if (epi == LM_ACT) return wide ? go<T, 4, 4, 4, LM_ACT>(g, nz, st) : go<T, 4, 2, 4, LM_ACT>(g, nz, st);
  }
  if (sizeof(T) == 2 && g.tile_rows == 64) {
    if (epi == LM_MOE_UP) return go<T, 4, 4, 4, LM_MOE_UP>(g, nz, st);
    if (epi == LM_MOE_DOWN) return go<T, 4, 4, 4, LM_MOE_DOWN>(g, nz, st);
  }
  // few rows and few features: one block of features per workgroup, so that more of the chip takes part
  if (few && (long)g.N * (g.max_tiles > 0 ? g.max_tiles : 1) <= 4096) {
    if (epi == LM_PROJ) return go<T, 1, 1, 16, LM_PROJ>(g, nz, st);
    if (epi == LM_ACT) return go<T, 1, 1, 16, LM_ACT>(g, nz, st);
    if (epi == LM_MOE_UP) return go<T, 1, 1, 16, LM_MOE_UP>(g, nz, st);
    if (epi == LM_MOE_DOWN) return go<T, 1, 1, 16, LM_MOE_DOWN>(g, nz, st);
  }
  switch (epi) {
    case LM_IN_ATTN: return few ? go<T, 1, 2, 8, LM_IN_ATTN>(g, nz, st) : go<T, 2, 2, 4, LM_IN_ATTN>(g, nz, st);
    case LM_IN_GRU_STEP: return go<T, 1, 3, 8, LM_IN_GRU_STEP>(g, nz, st);
    case LM_IN_GRU_SEQ: return few ? go<T, 1, 3, 8, LM_IN_GRU_SEQ>(g, nz, st) : go<T, 2, 3, 4, LM_IN_GRU_SEQ>(g, nz, st);
    case LM_OUT: return few ? go<T, 1, 1, 16, LM_OUT>(g, nz, st) : go<T, 2, 2, 4, LM_OUT>(g, nz, st);
    case LM_LOGITS: return few ? go<T, 1, 2, 8, LM_LOGITS>(g, nz, st) : go<T, 2, 2, 4, LM_LOGITS>(g, nz, st);
    case LM_HEAD: return few ? go<T, 1, 2, 8, LM_HEAD>(g, nz, st) : go<T, 2, 2, 4, LM_HEAD>(g, nz, st);
    case LM_PROJ: return few ? go<T, 1, 2, 8, LM_PROJ>(g, nz, st) : go<T, 2, 2, 4, LM_PROJ>(g, nz, st);
    case LM_PLAIN: return few ? go<T, 1, 1, 16, LM_PLAIN>(g, nz, st) : go<T, 2, 2, 4, LM_PLAIN>(g, nz, st);
    case LM_ACT: return few ? go<T, 1, 2, 8, LM_ACT>(g, nz, st) : go<T, 2, 2, 4, LM_ACT>(g, nz, st);
    case LM_MOE_UP: return few ? go<T, 1, 2, 8, LM_MOE_UP>(g, nz, st) : go<T, 2, 2, 4, LM_MOE_UP>(g, nz, st);
    case LM_MOE_DOWN: return few ? go<T, 1, 2, 8, LM_MOE_DOWN>(g, nz, st) : go<T, 2, 2, 4, LM_MOE_DOWN>(g, nz, st);
    case LM_EXPAND_K: return go<T, 2, 2, 4, LM_EXPAND_K>(g, nz, st);
    case LM_EXPAND_V: return go<T, 2, 2, 4, LM_EXPAND_V>(g, nz, st);
  }
  vui_set_error("lm gemm: unknown epilogue %d", epi);
  return VUI_EINVAL;
}

int launch_lm_gemm(int dtype, int epi, const LmGemm& g, int nz, hipStream_t st) {
  if (g.M < 1 || g.N < 16 || (g.N & 15) || g.K < 64 || (g.K & 63) || nz < 1) {
    vui_set_error("lm gemm: bad shape M=%d N=%d K=%d", g.M, g.N, g.K);
    return VUI_EINVAL;
  }
  const bool gru = epi == LM_IN_GRU_STEP || epi == LM_IN_GRU_SEQ;
  if ((gru && ((g.mix_blocks % 3) || (g.N / 16) % 3)) || (epi == LM_IN_ATTN && (g.mix_blocks % 2))) {
    vui_set_error("lm gemm: the input projection is not padded to its tile");
    return VUI_EINVAL;
  }
  if (epi == LM_IN_GRU_STEP && g.M > 16) { vui_set_error("lm gemm: a recurrence step takes at most 16 rows"); return VUI_EINVAL; }
  return dtype == VUI_DTYPE_F32 ? pick<float>(epi, g, nz, st) : pick<bf16_t>(epi, g, nz, st);
}

// ---- embedding rows: residual, operand copy, sums of squares per 16 columns ----
template <typename T>
__global__ __launch_bounds__(256) void lm_embed_kernel(const int64_t* tokens, const T* table, float* x, T* xt, float* ssq,
                                                       int width, int w64, int np, int vocab) {
  const int m = blockIdx.x, c = blockIdx.y * 256 + threadIdx.x;
  int64_t t = tokens[m];
  t = t < 0 ? 0 : (t >= vocab ? vocab - 1 : t);
  if (c < np * 16) {  // a multiple of 16: a 16-lane group is whole or absent
    const float v = c < width ? El<T>::ld(table + (size_t)t * width + c) : 0.f;
    x[(size_t)m * w64 + c] = v;
    El<T>::st(xt + tl_off<T>(m, c, w64), v);
    const float s = group16_sum(v * v);
    if ((c & 15) == 0) ssq[(size_t)m * np + (c >> 4)] = s;
  }
}
int launch_lm_embed(int dtype, const int64_t* tokens, const void* table, float* x, void* xt, float* ssq, int rows, int width,
                    int w64, int np, int vocab, hipStream_t st) {
  if (dtype == VUI_DTYPE_F32)
    hipLaunchKernelGGL(lm_embed_kernel<float>, dim3(rows, (np + 15) / 16), dim3(256), 0, st, tokens, (const float*)table, x, (float*)xt, ssq, width, w64, np, vocab);
  else
    hipLaunchKernelGGL(lm_embed_kernel<bf16_t>, dim3(rows, (np + 15) / 16), dim3(256), 0, st, tokens, (const bf16_t*)table, x, (bf16_t*)xt, ssq, width, w64, np, vocab);
  HIP_TRY(hipGetLastError());
  return VUI_OK;
}
