// Dense bf16 projections of the designs with a 32-bit residual stream, with what surrounds them
// in the same launch: the norm or the per-head norm and gate that makes their input in the head,
// the residual sum, the gated pair's activation or the soft cap in the tail.
//
// Decode widths (and 32-bit models at every width): a wavefront takes pairs of output rows over up
// to four activation rows; every workgroup makes the input rows itself (they are a few KB and come
// from the L2) while its first weights are on their way, as the k-quant mat-vec does with its norm
// (kq_qmv_kernel<.., PRE>). Every row of a call is summed exactly as it would be alone.
//
// Prefill widths (bf16): the input rows are made by a launch of their own, then one tiled GEMM on the
// matrix cores covers all matrices of the call.
#include "act_device.h"
#include "rt.h"

namespace {

constexpr int kSegs = 6;

struct RowsArgs {
  const void* x;
  const bf16_t* wn;
  const void* gate;
  float w_offset, eps, add_scale, soft_cap;
  int gate_act, pair_act;
  int head, M, K;
  int n;
  const bf16_t* w[kSegs];
  void* y[kSegs];
  int O[kSegs];
  int out[kSegs];
};

__device__ __forceinline__ float gate_of(int kind, float z) {
  const float s = dm_sigmoid_f32(z);
  return kind == ORNITH_GATE_SILU ? z * s : s;
}
__device__ __forceinline__ float pair_of(int kind, float gate, float up) {
  return (kind == ORNITH_PAIR_SILU ? gate * dm_sigmoid_f32(gate) : dm_gelu_tanh(gate)) * up;
}
// a sum as it is stored
__device__ __forceinline__ float stored(const RowsArgs& p, float v) {
  return p.soft_cap > 0.f ? p.soft_cap * dm_tanh(v / p.soft_cap) : v;
}
// four norm weights; none: ones
__device__ __forceinline__ void norm_weights(const bf16_t* w, float (&v)[4]) {
  v[0] = v[1] = v[2] = v[3] = 1.0f;
  if (w) act_load<4>(w, v);
}

// ---- decode widths ------------------------------------------------------------------------
constexpr int NT = 256, NR = 2, NU = 4;

// eight weights from 8j on; not VEC: rows of any length, past the end zero
template <bool VEC>
__device__ __forceinline__ uint4 weights8(const bf16_t* row, int j, int K) {
  if constexpr (VEC) return *reinterpret_cast<const uint4*>(row + 8 * j);
  uint32_t e[8];
#pragma unroll
  for (int i = 0; i < 8; ++i) e[i] = 8 * j + i < K ? row[8 * j + i] : 0;
  return make_uint4(e[0] | e[1] << 16, e[2] | e[3] << 16, e[4] | e[5] << 16, e[6] | e[7] << 16);
}

// the two weight rows of group g (a pair of output rows; with PAIR row g of both matrices)
template <bool PAIR>
__device__ __forceinline__ void group_rows(const RowsArgs& p, int g, const bf16_t* (&wr)[NR], int& seg, int& o) {
  if constexpr (PAIR) {
    seg = 0;
    o = g;
    wr[0] = p.w[0] + (size_t)g * p.K;
    wr[1] = p.w[1] + (size_t)g * p.K;
  } else {
    seg = 0;
    const bf16_t* w = p.w[0];
    int O = p.O[0];
#pragma unroll
    for (int i = 1; i < kSegs; ++i) {
      const int groups = (O + NR - 1) / NR;
      if (i < p.n && g >= groups) {
        g -= groups;
        w = p.w[i];
        O = p.O[i];
        seg = i;
      } else {
        break;
      }
    }
    o = g * NR;
    wr[0] = w + (size_t)o * p.K;
    wr[1] = w + (size_t)min(o + 1, O - 1) * p.K;
  }
}

// workgroup wg of `wgs` that share the call's groups of output rows
template <typename A, int MR, int PRE, bool PAIR, bool VEC>
__device__ __forceinline__ void dense_rows_body(const RowsArgs& p, int groups, int wg, int wgs) {
  extern __shared__ __attribute__((aligned(16))) char lds_raw[];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int K = p.K, K8 = (K + 7) / 8, Kp = K8 * 8;
  A* xs = reinterpret_cast<A*>(lds_raw);                              // [MR][Kp]
  float* aux = reinterpret_cast<float*>(lds_raw + (size_t)MR * Kp * sizeof(A));
  const int m0 = blockIdx.y * MR;
  const int stride = wgs * (NT / 64), nb = (K8 + 64 * NU - 1) / (64 * NU);
  int g = wg * (NT / 64) + wave;

  uint4 cur[NR][NU], nxt[NR][NU];
  const bf16_t* wr[NR];
  int seg = 0, o = 0;
  auto fetch = [&](int b, uint4 (&dst)[NR][NU]) {
#pragma unroll
    for (int u = 0; u < NU; ++u) {
      const int j = lane + 64 * (b * NU + u);
      if (j < K8) {
#pragma unroll
        for (int r = 0; r < NR; ++r) dst[r][u] = weights8<VEC>(wr[r], j, K);
      }
    }
  };

  // ---- the input rows --------------------------------------------------------------------
  if constexpr (PRE == ORNITH_PRE_NONE) {
    if (g < groups) {
      group_rows<PAIR>(p, g, wr, seg, o);
      fetch(0, cur);
    }
    for (int m = 0; m < MR; ++m) {
      const bool live = m0 + m < p.M;
      const A* src = reinterpret_cast<const A*>(p.x) + (size_t)(m0 + m) * K;
      if constexpr (VEC) {
        for (int c = tid; c < K8; c += NT) {
          float v[8] = {};
          if (live) act_load<8>(src + 8 * c, v);
          if constexpr (sizeof(A) == 2) {
            *reinterpret_cast<uint4*>(&xs[m * Kp + 8 * c]) =
                make_uint4(dm_f2bf2(v[0], v[1]), dm_f2bf2(v[2], v[3]), dm_f2bf2(v[4], v[5]), dm_f2bf2(v[6], v[7]));
          } else {
#pragma unroll
            for (int i = 0; i < 8; ++i) xs[m * Kp + 8 * c + i] = act_of<A>(v[i]);
          }
        }
      } else {
        for (int i = tid; i < Kp; i += NT) xs[m * Kp + i] = live && i < K ? src[i] : A(0);
      }
    }
  } else if constexpr (VEC) {
    // four consecutive values a thread and step; the first PC steps of every row stay in registers
    constexpr int PC = MR == 1 ? 8 : 4;
    float4 xr[MR][PC];
    const float* xsrc = reinterpret_cast<const float*>(p.x);
#pragma unroll
    for (int m = 0; m < MR; ++m)
#pragma unroll
      for (int c = 0; c < PC; ++c) {
        const int i = 4 * (tid + NT * c);
        xr[m][c] = make_float4(0.f, 0.f, 0.f, 0.f);
        if (m0 + m < p.M && i < K) xr[m][c] = *reinterpret_cast<const float4*>(xsrc + (size_t)(m0 + m) * K + i);
      }
    // (the rows above hit in cache: the cold weights are asked for behind them)
    if (g < groups) {
      group_rows<PAIR>(p, g, wr, seg, o);
      fetch(0, cur);
    }
    auto value = [&](int m, int c, int i) -> float4 {
      if (c < PC) return xr[m][c];
      if (m0 + m >= p.M) return make_float4(0.f, 0.f, 0.f, 0.f);
      return *reinterpret_cast<const float4*>(xsrc + (size_t)(m0 + m) * K + i);
    };
    auto square = [](const float4& v, float a) { return dm_fma(v.w, v.w, dm_fma(v.z, v.z, dm_fma(v.y, v.y, dm_fma(v.x, v.x, a)))); };
    if constexpr (PRE == ORNITH_PRE_NORM) {
#pragma unroll
      for (int m = 0; m < MR; ++m) {
        float a = 0.f;
#pragma unroll
        for (int c = 0; c < PC; ++c) a = square(xr[m][c], a);
        for (int c = PC; 4 * (tid + NT * c) < K; ++c) a = square(value(m, c, 4 * (tid + NT * c)), a);
        a = dm_wave_sum<64>(a);
        if (lane == 0) aux[m * 4 + wave] = a;
      }
      __syncthreads();
    } else {
      // sums of squares of four values, then of every head by sixteen lanes
      float* part = aux;                       // [MR][K/4]
      float* inv = aux + (size_t)MR * (K / 4); // [MR][K/head]
      const int heads = K / p.head, per = p.head / 4;
#pragma unroll
      for (int m = 0; m < MR; ++m) {
#pragma unroll
        for (int c = 0; c < PC; ++c)
          if (4 * (tid + NT * c) < K) part[m * (K / 4) + tid + NT * c] = square(xr[m][c], 0.f);
        for (int c = PC; 4 * (tid + NT * c) < K; ++c)
          part[m * (K / 4) + tid + NT * c] = square(value(m, c, 4 * (tid + NT * c)), 0.f);
      }
      __syncthreads();
      for (int h = tid >> 4; h < MR * heads; h += NT / 16) {
        float a = 0.f;
        for (int i = tid & 15; i < per; i += 16) a += part[h * per + i];
        a = dm_wave_sum<16>(a);
        if ((tid & 15) == 0) inv[h] = dm_rsqrt(a / (float)p.head + p.eps);
      }
      __syncthreads();
    }
#pragma unroll
    for (int m = 0; m < MR; ++m) {
      float rinv = 0.f;
      if constexpr (PRE == ORNITH_PRE_NORM)
        rinv = dm_rsqrt((((aux[m * 4] + aux[m * 4 + 1]) + aux[m * 4 + 2]) + aux[m * 4 + 3]) / (float)K + p.eps);
      auto emit = [&](int c) {
        const int i = 4 * (tid + NT * c);
        if (i >= K) return;
        const float4 x4 = value(m, c, i);
        float v[4] = {x4.x, x4.y, x4.z, x4.w}, wv[4];
        norm_weights(p.wn ? p.wn + i : nullptr, wv);
        if constexpr (PRE == ORNITH_PRE_NORM) {
#pragma unroll
          for (int e = 0; e < 4; ++e) v[e] = (v[e] * rinv) * (p.w_offset + wv[e]);
        } else {
          const float hinv = (aux + (size_t)MR * (K / 4))[m * (K / p.head) + i / p.head];
          float gv[4] = {};
          if (m0 + m < p.M) act_load<4>(reinterpret_cast<const A*>(p.gate) + (size_t)(m0 + m) * K + i, gv);
#pragma unroll
          for (int e = 0; e < 4; ++e) v[e] = ((v[e] * hinv) * wv[e]) * gate_of(p.gate_act, gv[e]);
        }
        act_store4(&xs[m * Kp + i], v);
      };
#pragma unroll
      for (int c = 0; c < PC; ++c) emit(c);
      for (int c = PC; 4 * (tid + NT * c) < K; ++c) emit(c);
    }
  } else {
    // any width: one row and one head after the other
    if (g < groups) {
      group_rows<PAIR>(p, g, wr, seg, o);
      fetch(0, cur);
    }
    const int head = PRE == ORNITH_PRE_NORM ? K : p.head;
    for (int m = 0; m < MR; ++m) {
      const bool live = m0 + m < p.M;
      const float* src = reinterpret_cast<const float*>(p.x) + (size_t)(m0 + m) * K;
      const A* gsrc = reinterpret_cast<const A*>(p.gate) + (size_t)(m0 + m) * K;
      for (int h0 = 0; h0 < K; h0 += head) {
        float a = 0.f;
        for (int i = tid; i < head; i += NT) {
          const float v = live ? src[h0 + i] : 0.f;
          a = dm_fma(v, v, a);
        }
        a = dm_wave_sum<64>(a);
        __syncthreads();
        if (lane == 0) aux[wave] = a;
        __syncthreads();
        const float rinv = dm_rsqrt((((aux[0] + aux[1]) + aux[2]) + aux[3]) / (float)head + p.eps);
        for (int i = tid; i < head; i += NT) {
          float v = live ? src[h0 + i] * rinv : 0.f;
          const float wv = p.wn ? dm_bf2f(p.wn[h0 + i]) : 1.0f;
          if constexpr (PRE == ORNITH_PRE_NORM) v = v * (p.w_offset + wv);
          else v = (v * wv) * gate_of(p.gate_act, live ? act_f(gsrc[h0 + i]) : 0.f);
          xs[m * Kp + h0 + i] = act_of<A>(v);
        }
      }
      for (int i = K + tid; i < Kp; i += NT) xs[m * Kp + i] = A(0);
    }
  }
  __syncthreads();

  // ---- row dots ------------------------------------------------------------------------------
  while (g < groups) {
    float acc[NR][MR];
#pragma unroll
    for (int r = 0; r < NR; ++r)
#pragma unroll
      for (int m = 0; m < MR; ++m) acc[r][m] = 0.f;
    const int seg_now = seg, o_now = o, gn = g + stride;
    for (int b = 0; b < nb; ++b) {
      if (b + 1 < nb) {
        fetch(b + 1, nxt);
      } else if (gn < groups) {
        group_rows<PAIR>(p, gn, wr, seg, o);
        fetch(0, nxt);
      }
#pragma unroll
      for (int u = 0; u < NU; ++u) {
        const int j = lane + 64 * (b * NU + u);
        if (j < K8) {
          float wv[NR][8];
#pragma unroll
          for (int r = 0; r < NR; ++r) {
            const uint4 q = cur[r][u];
            wv[r][0] = dm_bf2f_lo(q.x); wv[r][1] = dm_bf2f_hi(q.x); wv[r][2] = dm_bf2f_lo(q.y); wv[r][3] = dm_bf2f_hi(q.y);
            wv[r][4] = dm_bf2f_lo(q.z); wv[r][5] = dm_bf2f_hi(q.z); wv[r][6] = dm_bf2f_lo(q.w); wv[r][7] = dm_bf2f_hi(q.w);
          }
#pragma unroll
          for (int m = 0; m < MR; ++m) {
            float xv[8];
            act_load<8>(&xs[m * Kp + 8 * j], xv);
#pragma unroll
            for (int r = 0; r < NR; ++r)
#pragma unroll
              for (int i = 0; i < 8; ++i) acc[r][m] = dm_fma(wv[r][i], xv[i], acc[r][m]);
          }
        }
      }
#pragma unroll
      for (int r = 0; r < NR; ++r)
#pragma unroll
        for (int u = 0; u < NU; ++u) cur[r][u] = nxt[r][u];
    }
    float v[NR][MR];
#pragma unroll
    for (int r = 0; r < NR; ++r)
#pragma unroll
      for (int m = 0; m < MR; ++m) v[r][m] = dm_wave_sum<64>(acc[r][m]);
    if (lane == 0) {
      int O = p.O[0], kind = p.out[0];
      void* y = p.y[0];
#pragma unroll
      for (int i = 1; i < kSegs; ++i)
        if (i == seg_now) {
          O = p.O[i];
          kind = p.out[i];
          y = p.y[i];
        }
#pragma unroll
      for (int m = 0; m < MR; ++m) {
        if (m0 + m >= p.M) continue;
        if constexpr (PAIR) {
          reinterpret_cast<A*>(y)[(size_t)(m0 + m) * O + o_now] = act_of<A>(pair_of(p.pair_act, v[0][m], v[1][m]));
        } else {
#pragma unroll
          for (int r = 0; r < NR; ++r) {
            if (o_now + r >= O) continue;
            const size_t at = (size_t)(m0 + m) * O + o_now + r;
            if (kind == ORNITH_OUT_ACT) reinterpret_cast<A*>(y)[at] = act_of<A>(stored(p, v[r][m]));
            else if (kind == ORNITH_OUT_F32) reinterpret_cast<float*>(y)[at] = stored(p, v[r][m]);
            else reinterpret_cast<float*>(y)[at] += p.add_scale * v[r][m];
          }
        }
      }
    }
    g = gn;
  }
}

template <typename A, int MR, int PRE, bool PAIR, bool VEC>
__global__ __launch_bounds__(NT) void dense_rows_kernel(RowsArgs p, int groups) {
  dense_rows_body<A, MR, PRE, PAIR, VEC>(p, groups, blockIdx.x, gridDim.x);
}

// Two calls that read the same rows, each through its norm: plain outputs, and a gated pair. The first
// `split` workgroups take the first.
template <typename A, int MR, bool VEC>
__global__ __launch_bounds__(NT) void dense_rows_duo_kernel(RowsArgs a, RowsArgs b, int groups_a, int groups_b, int split) {
  if ((int)blockIdx.x < split) dense_rows_body<A, MR, ORNITH_PRE_NORM, false, VEC>(a, groups_a, blockIdx.x, split);
  else dense_rows_body<A, MR, ORNITH_PRE_NORM, true, VEC>(b, groups_b, blockIdx.x - split, gridDim.x - split);
}

size_t rows_lds(int MR, int K, size_t es, int pre, int head, bool vec) {
  const size_t Kp = (size_t)(K + 7) / 8 * 8;
  size_t aux = 16;
  if (pre == ORNITH_PRE_HEADS && vec) aux = (size_t)MR * (K / 4 + K / head);
  return (size_t)MR * Kp * es + (aux < 16 ? 16 : aux) * 4;
}

template <typename A, int MR, int PRE, bool PAIR, bool VEC>
int launch_rows_kernel(ornith_ctx* ctx, const RowsArgs& p, int groups, size_t lds) {
  if (lds > 65536)
    ORN_HIP(hipFuncSetAttribute((const void*)dense_rows_kernel<A, MR, PRE, PAIR, VEC>,
                                hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds));
  const int wgs = (groups + NT / 64 - 1) / (NT / 64), cap = 3 * (ctx->compute_units > 0 ? ctx->compute_units : 256);
  hipLaunchKernelGGL((dense_rows_kernel<A, MR, PRE, PAIR, VEC>), dim3(wgs < cap ? wgs : cap, (p.M + MR - 1) / MR), dim3(NT),
                     lds, ctx->stream, p, groups);
  ORN_LAUNCH_CHECK("dense_rows_kernel");
  return ORNITH_OK;
}

template <typename A, int MR, int PRE, bool VEC>
int launch_rows_pair(ornith_ctx* ctx, const RowsArgs& p, int groups, size_t lds, bool pair) {
  if constexpr (PRE != ORNITH_PRE_HEADS)
    if (pair) return launch_rows_kernel<A, MR, PRE, true, VEC>(ctx, p, groups, lds);
  return launch_rows_kernel<A, MR, PRE, false, VEC>(ctx, p, groups, lds);
}

template <typename A, int MR, bool VEC>
int launch_rows_pre(ornith_ctx* ctx, const RowsArgs& p, int groups, size_t lds, int pre, bool pair) {
  switch (pre) {
    case ORNITH_PRE_NONE: return launch_rows_pair<A, MR, ORNITH_PRE_NONE, VEC>(ctx, p, groups, lds, pair);
    case ORNITH_PRE_NORM: return launch_rows_pair<A, MR, ORNITH_PRE_NORM, VEC>(ctx, p, groups, lds, pair);
    default: return launch_rows_pair<A, MR, ORNITH_PRE_HEADS, VEC>(ctx, p, groups, lds, false);
  }
}

int row_groups(const RowsArgs& p, bool pair) {
  if (pair) return p.O[0];
  int groups = 0;
  for (int i = 0; i < p.n; ++i) groups += (p.O[i] + NR - 1) / NR;
  return groups;
}

template <typename A, int MR, bool VEC>
int launch_duo_kernel(ornith_ctx* ctx, const RowsArgs& a, const RowsArgs& b, size_t lds) {
  if (lds > 65536)
    ORN_HIP(hipFuncSetAttribute((const void*)dense_rows_duo_kernel<A, MR, VEC>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds));
  constexpr int PER = NT / 64;
  const int ga = row_groups(a, false), gb = row_groups(b, true), cap = 3 * (ctx->compute_units > 0 ? ctx->compute_units : 256);
  int wa = (ga + PER - 1) / PER, wb = (gb + PER - 1) / PER;
  if (wa + wb > cap) {  // shares by their work; a group is two rows of either
    wa = (int)((long)cap * ga / (ga + gb));
    wa = wa < 1 ? 1 : wa > cap - 1 ? cap - 1 : wa;
    wb = cap - wa;
  }
  hipLaunchKernelGGL((dense_rows_duo_kernel<A, MR, VEC>), dim3(wa + wb, (a.M + MR - 1) / MR), dim3(NT), lds, ctx->stream, a, b, ga, gb,
                     wa);
  ORN_LAUNCH_CHECK("dense_rows_duo_kernel");
  return ORNITH_OK;
}

template <typename A>
int launch_duo(ornith_ctx* ctx, const RowsArgs& a, const RowsArgs& b) {
  const bool vec = a.K % 8 == 0;
  int MR = !vec ? 1 : a.M >= 3 ? 4 : a.M;
  while (MR > 1 && rows_lds(MR, a.K, sizeof(A), ORNITH_PRE_NORM, 0, vec) > 65536) MR /= 2;
  const size_t lds = rows_lds(MR, a.K, sizeof(A), ORNITH_PRE_NORM, 0, vec);
  ORN_REQUIRE(lds <= 160 * 1024, "dense_rows: rows of %d values do not fit a compute unit's local memory", a.K);
  if (!vec) return launch_duo_kernel<A, 1, false>(ctx, a, b, lds);
  switch (MR) {
    case 1: return launch_duo_kernel<A, 1, true>(ctx, a, b, lds);
    case 2: return launch_duo_kernel<A, 2, true>(ctx, a, b, lds);
    default: return launch_duo_kernel<A, 4, true>(ctx, a, b, lds);
  }
}

template <typename A>
int launch_rows(ornith_ctx* ctx, const RowsArgs& p, int pre, bool pair) {
  const int groups = row_groups(p, pair);
  const bool vec = p.K % 8 == 0 && (pre != ORNITH_PRE_HEADS || p.head % 4 == 0);
  int MR = !vec ? 1 : p.M >= 3 ? 4 : p.M;
  while (MR > 1 && rows_lds(MR, p.K, sizeof(A), pre, p.head, vec) > 65536) MR /= 2;
  const size_t lds = rows_lds(MR, p.K, sizeof(A), pre, p.head, vec);
  ORN_REQUIRE(lds <= 160 * 1024, "dense_rows: rows of %d values do not fit a compute unit's local memory", p.K);
  if (!vec) return launch_rows_pre<A, 1, false>(ctx, p, groups, lds, pre, pair);
  switch (MR) {
    case 1: return launch_rows_pre<A, 1, true>(ctx, p, groups, lds, pre, pair);
    case 2: return launch_rows_pre<A, 2, true>(ctx, p, groups, lds, pre, pair);
    default: return launch_rows_pre<A, 4, true>(ctx, p, groups, lds, pre, pair);
  }
}

// ---- the input rows as a launch of their own ---------------------------------------------------
// one workgroup a row: act(x / rms * (w_offset + w)), fp32 in
template <typename A>
__global__ __launch_bounds__(NT) void norm_rows_kernel(const float* x, const bf16_t* w, float w_offset, float eps, int n,
                                                       A* out) {
  __shared__ float red[4];
  const float* src = x + (size_t)blockIdx.x * n;
  A* dst = out + (size_t)blockIdx.x * n;
  const int tid = threadIdx.x;
  const bool vec = n % 4 == 0;
  constexpr int PC = 4;
  float4 xr[PC];
  float a = 0.f;
  if (vec) {
#pragma unroll
    for (int c = 0; c < PC; ++c) {
      const int i = 4 * (tid + NT * c);
      xr[c] = i < n ? *reinterpret_cast<const float4*>(src + i) : make_float4(0.f, 0.f, 0.f, 0.f);
    }
#pragma unroll
    for (int c = 0; c < PC; ++c) a = dm_fma(xr[c].w, xr[c].w, dm_fma(xr[c].z, xr[c].z, dm_fma(xr[c].y, xr[c].y, dm_fma(xr[c].x, xr[c].x, a))));
    for (int i = 4 * (tid + NT * PC); i < n; i += 4 * NT) {
      const float4 v = *reinterpret_cast<const float4*>(src + i);
      a = dm_fma(v.w, v.w, dm_fma(v.z, v.z, dm_fma(v.y, v.y, dm_fma(v.x, v.x, a))));
    }
  } else {
    for (int i = tid; i < n; i += NT) a = dm_fma(src[i], src[i], a);
  }
  a = dm_wave_sum<64>(a);
  if ((tid & 63) == 0) red[tid >> 6] = a;
  __syncthreads();
  const float inv = dm_rsqrt((((red[0] + red[1]) + red[2]) + red[3]) / (float)n + eps);
  if (vec) {
    auto emit = [&](const float4& x4, int i) {
      float wv[4];
      act_load<4>(w + i, wv);
      const float v[4] = {(x4.x * inv) * (w_offset + wv[0]), (x4.y * inv) * (w_offset + wv[1]),
                          (x4.z * inv) * (w_offset + wv[2]), (x4.w * inv) * (w_offset + wv[3])};
      act_store4(dst + i, v);
    };
#pragma unroll
    for (int c = 0; c < PC; ++c)
      if (4 * (tid + NT * c) < n) emit(xr[c], 4 * (tid + NT * c));
    for (int i = 4 * (tid + NT * PC); i < n; i += 4 * NT) emit(*reinterpret_cast<const float4*>(src + i), i);
  } else {
    for (int i = tid; i < n; i += NT) dst[i] = act_of<A>((src[i] * inv) * (w_offset + dm_bf2f(w[i])));
  }
}

// one wavefront a head of a row: act(x / rms_head * w * gate_act(gate))
template <typename A>
__global__ __launch_bounds__(NT) void head_norm_gate_kernel(const float* x, const bf16_t* w, const A* gate, int gate_act,
                                                            float eps, int heads, int head, int total, A* out) {
  const int hr = blockIdx.x * (NT / 64) + (threadIdx.x >> 6), lane = threadIdx.x & 63;
  if (hr >= total) return;
  const size_t base = (size_t)hr * head;
  const int w0 = (hr % heads) * head;
  float a = 0.f;
  if (head % 4 == 0) {
    for (int i = 4 * lane; i < head; i += 256) {
      const float4 v = *reinterpret_cast<const float4*>(x + base + i);
      a = dm_fma(v.w, v.w, dm_fma(v.z, v.z, dm_fma(v.y, v.y, dm_fma(v.x, v.x, a))));
    }
    const float inv = dm_rsqrt(dm_wave_sum<64>(a) / (float)head + eps);
    for (int i = 4 * lane; i < head; i += 256) {
      const float4 x4 = *reinterpret_cast<const float4*>(x + base + i);
      float wv[4], gv[4];
      norm_weights(w ? w + w0 + i : nullptr, wv);
      act_load<4>(gate + base + i, gv);
      const float v[4] = {((x4.x * inv) * wv[0]) * gate_of(gate_act, gv[0]), ((x4.y * inv) * wv[1]) * gate_of(gate_act, gv[1]),
                          ((x4.z * inv) * wv[2]) * gate_of(gate_act, gv[2]), ((x4.w * inv) * wv[3]) * gate_of(gate_act, gv[3])};
      act_store4(out + base + i, v);
    }
  } else {
    for (int i = lane; i < head; i += 64) a = dm_fma(x[base + i], x[base + i], a);
    const float inv = dm_rsqrt(dm_wave_sum<64>(a) / (float)head + eps);
    for (int i = lane; i < head; i += 64)
      out[base + i] = act_of<A>(((x[base + i] * inv) * (w ? dm_bf2f(w[w0 + i]) : 1.0f)) * gate_of(gate_act, act_f(gate[base + i])));
  }
}

// x = table[id] * scale, fp32: a workgroup takes 1024 values of a row
__global__ __launch_bounds__(NT) void embed_rows_kernel(const bf16_t* table, const uint32_t* ids, float scale, int V, int n,
                                                        float* out) {
  const bf16_t* src = table + (size_t)min(ids[blockIdx.y], (uint32_t)(V - 1)) * n;
  float* dst = out + (size_t)blockIdx.y * n;
  const int i = 4 * (blockIdx.x * NT + threadIdx.x);
  if (n % 4 == 0) {
    if (i >= n) return;
    float v[4];
    act_load<4>(src + i, v);
#pragma unroll
    for (int e = 0; e < 4; ++e) v[e] *= scale;
    act_store4(dst + i, v);
  } else {
    for (int e = i; e < min(i + 4, n); ++e) dst[e] = dm_bf2f(src[e]) * scale;
  }
}

// x = table[id] / rms * (w_offset + w), fp32: a workgroup a row
__global__ __launch_bounds__(NT) void embed_norm_rows_kernel(const bf16_t* table, const uint32_t* ids, int V, int n,
                                                             const bf16_t* w, float w_offset, float eps, float* out) {
  __shared__ float red[4];
  const bf16_t* src = table + (size_t)min(ids[blockIdx.x], (uint32_t)(V - 1)) * n;
  float* dst = out + (size_t)blockIdx.x * n;
  const int tid = threadIdx.x;
  constexpr int PC = 4;
  const bool vec = n % 8 == 0;
  float x[PC][8];
  float a = 0.f;
  if (vec) {
#pragma unroll
    for (int c = 0; c < PC; ++c) {
      const int i = 8 * (tid + NT * c);
#pragma unroll
      for (int e = 0; e < 8; ++e) x[c][e] = 0.f;
      if (i < n) act_load<8>(src + i, x[c]);
    }
#pragma unroll
    for (int c = 0; c < PC; ++c)
#pragma unroll
      for (int e = 0; e < 8; ++e) a = dm_fma(x[c][e], x[c][e], a);
  }
  for (int i = vec ? 8 * NT * PC + tid : tid; i < n; i += NT) {
    const float v = dm_bf2f(src[i]);
    a = dm_fma(v, v, a);
  }
  a = dm_wave_sum<64>(a);
  if ((tid & 63) == 0) red[tid >> 6] = a;
  __syncthreads();
  const float inv = dm_rsqrt((((red[0] + red[1]) + red[2]) + red[3]) / (float)n + eps);
  if (vec) {
#pragma unroll
    for (int c = 0; c < PC; ++c) {
      const int i = 8 * (tid + NT * c);
      if (i >= n) continue;
      float wv[8];
      act_load<8>(w + i, wv);
#pragma unroll
      for (int h = 0; h < 2; ++h) {
        float v[4];
#pragma unroll
        for (int e = 0; e < 4; ++e) v[e] = (x[c][4 * h + e] * inv) * (w_offset + wv[4 * h + e]);
        act_store4(dst + i + 4 * h, v);
      }
    }
  }
  for (int i = vec ? 8 * NT * PC + tid : tid; i < n; i += NT) dst[i] = (dm_bf2f(src[i]) * inv) * (w_offset + dm_bf2f(w[i]));
}

__global__ __launch_bounds__(NT) void round_bf16_kernel(const float* x, size_t n, bf16_t* out) {
  for (size_t i = (size_t)blockIdx.x * NT + threadIdx.x; i < n; i += (size_t)gridDim.x * NT) out[i] = dm_f2bf(x[i]);
}

// ---- prefill widths: tiled GEMM on the matrix cores ---------------------------------------------
// y[M, O] = x[M, K] . W[O, K]^T. The weights are the first operand, so a lane ends up with four
// consecutive output features of one token. K goes through LDS in slabs of 64: double buffered,
// 16-byte pieces placed at piece ^ (row / 2 mod 8), which spreads both the writes and the fragment
// reads over all banks; the next slab's pieces wait in registers while this one is multiplied.
typedef __bf16 g_bf16x8 __attribute__((ext_vector_type(8)));
typedef float g_f32x16 __attribute__((ext_vector_type(16)));
typedef uint32_t g_u32x4 __attribute__((ext_vector_type(4)));

template <int BM, int BN, bool PAIR>
__global__ __launch_bounds__(256) void dense_gemm_kernel(RowsArgs p, int tiles_n, int tiles_m, int per_die) {
  constexpr int BK = 64, MT = BM / 64, NTL = BN / 64;
  static_assert(!PAIR || NTL == 2, "gate and up tiles of a wavefront");
  __shared__ __attribute__((aligned(16))) bf16_t Xs[2][BM * BK];
  __shared__ __attribute__((aligned(16))) bf16_t Ws[2][BN * BK];
  // consecutive workgroups run on different dies: give each die a contiguous run of tiles, and walk
  // the run in blocks of eight token tiles so that a die's cache keeps both operands
  const int id = (blockIdx.x & 7) * per_die + (blockIdx.x >> 3);
  if (id >= tiles_n * tiles_m) return;
  constexpr int GM = 8;
  const int band = id / (GM * tiles_n), in = id % (GM * tiles_n), bm = min(GM, tiles_m - band * GM);
  const int tm = band * GM + in % bm, tn = in / bm;
  const int K = p.K, m0 = tm * BM;
  // the matrix this column tile belongs to
  int seg = 0, t = tn;
  if constexpr (!PAIR) {
#pragma unroll
    for (int i = 0; i < kSegs - 1; ++i) {
      const int tiles = (p.O[seg] + BN - 1) / BN;
      if (seg + 1 < p.n && t >= tiles) {
        t -= tiles;
        ++seg;
      }
    }
  }
  const int O = p.O[seg], n0 = t * (PAIR ? BN / 2 : BN);

  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, l32 = lane & 31, lh = lane >> 5;
  const int wm = wave & 1, wn = wave >> 1;
  constexpr int XL = BM / 32, WL = BN / 32;
  const int piece = tid & 7, row8 = tid >> 3;
  const bf16_t* xp[XL];
  const bf16_t* wp[WL];
  int xl[XL], wl[WL];
#pragma unroll
  for (int i = 0; i < XL; ++i) {
    const int r = row8 + 32 * i;
    xp[i] = reinterpret_cast<const bf16_t*>(p.x) + (size_t)min(m0 + r, p.M - 1) * K + 8 * piece;
    xl[i] = r * BK + 8 * (piece ^ ((r >> 1) & 7));
  }
#pragma unroll
  for (int i = 0; i < WL; ++i) {
    const int r = row8 + 32 * i;
    if constexpr (PAIR) {
      const int f = n0 + (r / 64) * 32 + (r & 31);
      wp[i] = p.w[(r >> 5) & 1] + (size_t)min(f, O - 1) * K + 8 * piece;
    } else {
      wp[i] = p.w[seg] + (size_t)min(n0 + r, O - 1) * K + 8 * piece;
    }
    wl[i] = r * BK + 8 * (piece ^ ((r >> 1) & 7));
  }
  g_u32x4 xr[XL], wr[WL];
  auto load = [&](int k0) {
    const bool in_k = k0 + 8 * piece < K;  // K is a multiple of 8
    const g_u32x4 zero = {0, 0, 0, 0};
#pragma unroll
    for (int i = 0; i < XL; ++i) xr[i] = in_k ? *reinterpret_cast<const g_u32x4*>(xp[i] + k0) : zero;
#pragma unroll
    for (int i = 0; i < WL; ++i) wr[i] = in_k ? *reinterpret_cast<const g_u32x4*>(wp[i] + k0) : zero;
  };
  auto store = [&](int buf) {
#pragma unroll
    for (int i = 0; i < XL; ++i) *reinterpret_cast<g_u32x4*>(&Xs[buf][xl[i]]) = xr[i];
#pragma unroll
    for (int i = 0; i < WL; ++i) *reinterpret_cast<g_u32x4*>(&Ws[buf][wl[i]]) = wr[i];
  };
  g_f32x16 acc[NTL][MT];
#pragma unroll
  for (int a = 0; a < NTL; ++a)
#pragma unroll
    for (int b = 0; b < MT; ++b)
#pragma unroll
      for (int i = 0; i < 16; ++i) acc[a][b][i] = 0.f;

  const int slabs = (K + BK - 1) / BK;
  load(0);
  store(0);
  if (slabs > 1) load(BK);
  __syncthreads();
  for (int s = 0; s < slabs; ++s) {
    const int buf = s & 1;
#pragma unroll
    for (int kk = 0; kk < 4; ++kk) {
      g_bf16x8 wf[NTL], xf[MT];
#pragma unroll
      for (int a = 0; a < NTL; ++a) {
        const int r = wn * (BN / 2) + a * 32 + l32;
        wf[a] = *reinterpret_cast<const g_bf16x8*>(&Ws[buf][r * BK + 8 * ((2 * kk + lh) ^ ((r >> 1) & 7))]);
      }
#pragma unroll
      for (int b = 0; b < MT; ++b) {
        const int r = wm * (BM / 2) + b * 32 + l32;
        xf[b] = *reinterpret_cast<const g_bf16x8*>(&Xs[buf][r * BK + 8 * ((2 * kk + lh) ^ ((r >> 1) & 7))]);
      }
#pragma unroll
      for (int a = 0; a < NTL; ++a)
#pragma unroll
        for (int b = 0; b < MT; ++b) acc[a][b] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(wf[a], xf[b], acc[a][b], 0, 0, 0);
    }
    if (s + 1 < slabs) {
      store(buf ^ 1);
      if (s + 2 < slabs) load((s + 2) * BK);
    }
    __syncthreads();
  }
  // D[feature 8q + 4 lh + e][token l32] is element 4q + e
  const int kind = p.out[seg];
  void* y = p.y[seg];
#pragma unroll
  for (int b = 0; b < MT; ++b) {
    const int m = m0 + wm * (BM / 2) + b * 32 + l32;
    if (m >= p.M) continue;
#pragma unroll
    for (int a = 0; a < (PAIR ? 1 : NTL); ++a)
#pragma unroll
      for (int q = 0; q < 4; ++q) {
        float v[4];
        int f;
        if constexpr (PAIR) {
          f = n0 + wn * 32 + 8 * q + 4 * lh;
#pragma unroll
          for (int e = 0; e < 4; ++e) v[e] = pair_of(p.pair_act, acc[0][b][4 * q + e], acc[NTL - 1][b][4 * q + e]);
        } else {
          f = n0 + wn * (BN / 2) + a * 32 + 8 * q + 4 * lh;
#pragma unroll
          for (int e = 0; e < 4; ++e) v[e] = kind == ORNITH_OUT_ADD ? p.add_scale * acc[a][b][4 * q + e] : stored(p, acc[a][b][4 * q + e]);
        }
        const size_t at = (size_t)m * O + f;
        if (f + 3 < O && (O & 3) == 0) {
          if (kind == ORNITH_OUT_ACT) {
            act_store4(reinterpret_cast<bf16_t*>(y) + at, v);
          } else {
            float* yf = reinterpret_cast<float*>(y) + at;
            if (kind == ORNITH_OUT_ADD) {
              float old[4];
              act_load<4>(yf, old);
#pragma unroll
              for (int e = 0; e < 4; ++e) v[e] = old[e] + v[e];
            }
            act_store4(yf, v);
          }
        } else {
#pragma unroll
          for (int e = 0; e < 4; ++e)
            if (f + e < O) {
              if (kind == ORNITH_OUT_ACT) reinterpret_cast<bf16_t*>(y)[at + e] = dm_f2bf(v[e]);
              else if (kind == ORNITH_OUT_F32) reinterpret_cast<float*>(y)[at + e] = v[e];
              else reinterpret_cast<float*>(y)[at + e] += v[e];
            }
        }
      }
  }
}

template <int BM, int BN, bool PAIR>
int launch_gemm_tile(ornith_ctx* ctx, const RowsArgs& p) {
  int tiles_n = 0;
  if (PAIR) tiles_n = (p.O[0] + BN / 2 - 1) / (BN / 2);
  else for (int i = 0; i < p.n; ++i) tiles_n += (p.O[i] + BN - 1) / BN;
  const int tiles_m = (p.M + BM - 1) / BM, per_die = (tiles_n * tiles_m + 7) / 8;
  hipLaunchKernelGGL((dense_gemm_kernel<BM, BN, PAIR>), dim3(8 * per_die), dim3(256), 0, ctx->stream, p, tiles_n, tiles_m,
                     per_die);
  ORN_LAUNCH_CHECK("dense_gemm_kernel");
  return ORNITH_OK;
}

int launch_gemm(ornith_ctx* ctx, const RowsArgs& p, bool pair) {
  long cols = 0;
  for (int i = 0; i < p.n; ++i) cols += p.O[i];
  const long tiles = (cols + 127) / 128 * ((p.M + 127) / 128);
  const bool big = tiles >= (ctx->compute_units > 0 ? ctx->compute_units : 256);
  if (pair) return big ? launch_gemm_tile<128, 128, true>(ctx, p) : launch_gemm_tile<64, 128, true>(ctx, p);
  return big ? launch_gemm_tile<128, 128, false>(ctx, p) : launch_gemm_tile<64, 64, false>(ctx, p);
}

}  // namespace

extern "C" {

int ornith_norm_rows(ornith_ctx* ctx, const float* d_x, const void* d_w, float w_offset, int rows, int n, float eps, int act,
                     void* d_out) {
  ORN_REQUIRE(ctx && d_x && d_w && d_out, "norm_rows: null argument");
  ORN_REQUIRE(rows >= 1 && n >= 1, "norm_rows: rows=%d n=%d", rows, n);
  if (act == ORNITH_F32)
    hipLaunchKernelGGL(norm_rows_kernel<float>, dim3(rows), dim3(NT), 0, ctx->stream, d_x, (const bf16_t*)d_w, w_offset, eps, n,
                       (float*)d_out);
  else
    hipLaunchKernelGGL(norm_rows_kernel<bf16_t>, dim3(rows), dim3(NT), 0, ctx->stream, d_x, (const bf16_t*)d_w, w_offset, eps, n,
                       (bf16_t*)d_out);
  ORN_LAUNCH_CHECK("norm_rows_kernel");
  return ORNITH_OK;
}

int ornith_head_norm_gate(ornith_ctx* ctx, const float* d_x, const void* d_w, const void* d_gate, int gate_act, int rows,
                          int heads, int head, float eps, int act, void* d_out) {
  ORN_REQUIRE(ctx && d_x && d_gate && d_out, "head_norm_gate: null argument");
  ORN_REQUIRE(rows >= 1 && heads >= 1 && head >= 1, "head_norm_gate: rows=%d heads=%d of %d", rows, heads, head);
  const int total = rows * heads, wgs = (total + NT / 64 - 1) / (NT / 64);
  if (act == ORNITH_F32)
    hipLaunchKernelGGL(head_norm_gate_kernel<float>, dim3(wgs), dim3(NT), 0, ctx->stream, d_x, (const bf16_t*)d_w,
                       (const float*)d_gate, gate_act, eps, heads, head, total, (float*)d_out);
  else
    hipLaunchKernelGGL(head_norm_gate_kernel<bf16_t>, dim3(wgs), dim3(NT), 0, ctx->stream, d_x, (const bf16_t*)d_w,
                       (const bf16_t*)d_gate, gate_act, eps, heads, head, total, (bf16_t*)d_out);
  ORN_LAUNCH_CHECK("head_norm_gate_kernel");
  return ORNITH_OK;
}

int ornith_embed_rows(ornith_ctx* ctx, const ornith_linear* table, const uint32_t* d_ids, int n, float scale, float* d_out) {
  ORN_REQUIRE(ctx && table && d_ids && d_out, "embed_rows: null argument");
  ORN_REQUIRE(table->mode == ORNITH_LIN_DENSE && table->d_w && n >= 1 && n <= 65535, "embed_rows: table mode %d, n=%d", table->mode, n);
  hipLaunchKernelGGL(embed_rows_kernel, dim3((table->K + 4 * NT - 1) / (4 * NT), n), dim3(NT), 0, ctx->stream, (const bf16_t*)table->d_w, d_ids, scale, table->O,
                     table->K, d_out);
  ORN_LAUNCH_CHECK("embed_rows_kernel");
  return ORNITH_OK;
}

int ornith_embed_norm_rows(ornith_ctx* ctx, const ornith_linear* table, const uint32_t* d_ids, int n, const void* d_w,
                           float w_offset, float eps, float* d_out) {
  ORN_REQUIRE(ctx && table && d_ids && d_w && d_out, "embed_norm_rows: null argument");
  ORN_REQUIRE(table->mode == ORNITH_LIN_DENSE && table->d_w && n >= 1, "embed_norm_rows: table mode %d, n=%d", table->mode, n);
  hipLaunchKernelGGL(embed_norm_rows_kernel, dim3(n), dim3(NT), 0, ctx->stream, (const bf16_t*)table->d_w, d_ids, table->O, table->K,
                     (const bf16_t*)d_w, w_offset, eps, d_out);
  ORN_LAUNCH_CHECK("embed_norm_rows_kernel");
  return ORNITH_OK;
}

int ornith_round_bf16(ornith_ctx* ctx, const float* d_x, size_t n, void* d_out) {
  ORN_REQUIRE(ctx && d_x && d_out && n >= 1, "round_bf16: null argument");
  const size_t wgs = (n + NT - 1) / NT;
  hipLaunchKernelGGL(round_bf16_kernel, dim3((unsigned)(wgs < 4096 ? wgs : 4096)), dim3(NT), 0, ctx->stream, d_x, n, (bf16_t*)d_out);
  ORN_LAUNCH_CHECK("round_bf16_kernel");
  return ORNITH_OK;
}

static int rows_args(ornith_ctx* ctx, const ornith_dense_call* c, RowsArgs& p) {
  ORN_REQUIRE(ctx && c && c->d_x, "dense_rows: null argument");
  ORN_REQUIRE(c->act == ORNITH_BF16 || c->act == ORNITH_F32, "dense_rows: activation type %d", c->act);
  ORN_REQUIRE(c->M >= 1 && c->K >= 1 && c->n >= 1 && c->n <= kSegs, "dense_rows: M=%d K=%d n=%d", c->M, c->K, c->n);
  ORN_REQUIRE(c->pre >= ORNITH_PRE_NONE && c->pre <= ORNITH_PRE_HEADS, "dense_rows: prologue %d", c->pre);
  ORN_REQUIRE(c->pre != ORNITH_PRE_NORM || c->d_norm_w, "dense_rows: norm weight missing");
  ORN_REQUIRE(c->pre != ORNITH_PRE_HEADS || (c->d_gate && c->head_dim >= 1 && c->K % c->head_dim == 0 && !c->pair_act),
              "dense_rows: heads of %d in rows of %d", c->head_dim, c->K);
  p = RowsArgs{};
  p.x = c->d_x;
  p.wn = (const bf16_t*)c->d_norm_w;
  p.gate = c->d_gate;
  p.w_offset = c->w_offset;
  p.eps = c->eps;
  p.add_scale = c->add_scale;
  p.soft_cap = c->soft_cap;
  p.gate_act = c->gate_act;
  p.pair_act = c->pair_act;
  p.head = c->head_dim;
  p.M = c->M;
  p.K = c->K;
  p.n = c->n;
  for (int i = 0; i < c->n; ++i) {
    const ornith_linear* w = c->w[i];
    ORN_REQUIRE(w && w->d_w, "dense_rows: matrix %d missing", i);
    ORN_REQUIRE(w->mode == ORNITH_LIN_DENSE && w->K == c->K && w->O >= 1, "dense_rows: matrix %d is [%d,%d], rows have %d", i,
                w->O, w->K, c->K);
    ORN_REQUIRE(c->out[i] >= ORNITH_OUT_ACT && c->out[i] <= ORNITH_OUT_ADD, "dense_rows: output kind %d", c->out[i]);
    p.w[i] = (const bf16_t*)w->d_w;
    p.O[i] = w->O;
    p.y[i] = c->d_y[i];
    p.out[i] = c->out[i];
    ORN_REQUIRE(c->d_y[i] || (c->pair_act && i == 1), "dense_rows: output %d missing", i);
  }
  ORN_REQUIRE(!c->pair_act || (c->n == 2 && p.O[0] == p.O[1]), "dense_rows: a gated pair is two matrices of one size");
  ORN_REQUIRE(c->K % 8 != 0 || (((uintptr_t)c->d_x | (uintptr_t)c->d_gate) & 15) == 0, "dense_rows: operands must be 16-byte aligned");
  return ORNITH_OK;
}

static bool runs_as_gemm(const ornith_dense_call* c) { return c->act == ORNITH_BF16 && c->M >= kPrefillRows && c->K % 8 == 0; }

int ornith_dense_rows_duo(ornith_ctx* ctx, const ornith_dense_call* a, const ornith_dense_call* b) {
  RowsArgs p, q;
  int rc = rows_args(ctx, a, p);
  if (!rc) rc = rows_args(ctx, b, q);
  if (rc) return rc;
  ORN_REQUIRE(a->act == b->act && a->M == b->M && a->K == b->K && a->pre == ORNITH_PRE_NORM && b->pre == ORNITH_PRE_NORM &&
                  !a->pair_act && b->pair_act,
              "dense_rows_duo: normed rows [%d,%d] for plain outputs beside normed rows [%d,%d] for a gated pair", a->M, a->K, b->M, b->K);
  if (!runs_as_gemm(a)) return a->act == ORNITH_F32 ? launch_duo<float>(ctx, p, q) : launch_duo<bf16_t>(ctx, p, q);
  rc = ornith_dense_rows(ctx, a);
  return rc ? rc : ornith_dense_rows(ctx, b);
}

int ornith_dense_rows(ornith_ctx* ctx, const ornith_dense_call* c) {
  RowsArgs p;
  int rc = rows_args(ctx, c, p);
  if (rc) return rc;
  if (!runs_as_gemm(c))
    return c->act == ORNITH_F32 ? launch_rows<float>(ctx, p, c->pre, c->pair_act != ORNITH_PAIR_NONE)
                                : launch_rows<bf16_t>(ctx, p, c->pre, c->pair_act != ORNITH_PAIR_NONE);
  if (c->pre != ORNITH_PRE_NONE) {
    ORN_REQUIRE(c->d_rows, "dense_rows: %d rows need the buffer for the rows the matrices read", c->M);
    rc = c->pre == ORNITH_PRE_NORM
                       ? ornith_norm_rows(ctx, (const float*)c->d_x, c->d_norm_w, c->w_offset, c->M, c->K, c->eps, c->act, c->d_rows)
                       : ornith_head_norm_gate(ctx, (const float*)c->d_x, c->d_norm_w, c->d_gate, c->gate_act, c->M,
                                               c->K / c->head_dim, c->head_dim, c->eps, c->act, c->d_rows);
    if (rc) return rc;
    p.x = c->d_rows;
  }
  return launch_gemm(ctx, p, c->pair_act != ORNITH_PAIR_NONE);
}

}  // extern "C"
