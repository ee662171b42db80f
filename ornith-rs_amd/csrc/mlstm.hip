// mLSTM: a matrix memory per head, S (value x key channels), with exponential input gates and a running
// maximum m that keeps them in range (Beck et al., "xLSTM: Extended Long Short-Term Memory"). The
// arithmetic is stated at ornith_mlstm in ornith_hip.h. The state of a head in memory, fp32:
//   S [vdim][ds], n [ds], m, with ds = dim rounded up to 4 (the padding stays zero).
//
// Token by token (decode widths, 32-bit models): a workgroup takes sixteen value channels of one head,
// sixteen lanes a channel, the state in registers across the call's tokens. Every workgroup walks the
// normaliser n and m for itself, so a call never writes the slot it started from.
//
// In chunks of 64 tokens (prefill widths, bf16), three launches. With F_t the sum of the log forget
// gates of a chunk up to t and m_0, S_0, n_0 what the chunk starts from,
//   m_t  = F_t + max(m_0, max_{s<=t} (i_s - F_s))
//   num_t = e^(F_t + m_0 - m_t) S_0 q_t + sum_{s<=t} P_ts v_s,  P_ts = e^(F_t - F_s + i_s - m_t) (q_t . k_s)
//   den_t = the same with n_0 and 1 in place of S_0 and v_s
//   S_C  = e^(F_C + m_0 - m_C) S_0 + sum_s e^(F_C - F_s + i_s - m_C) v_s k_s^T
// (every exponent is at most 0): mlstm_gates_kernel makes the gates, m and the weights of every token;
// mlstm_scan_kernel walks S from chunk to chunk, tile by tile independent, leaving each chunk's S_0 and
// n_0; mlstm_out_kernel makes the outputs, all chunks at once. q, k, v are bf16 numbers; S_0, P and the
// weighted keys go to the matrix cores as two bf16 parts each, so nothing of the recurrence is rounded to bf16.
#include "act_device.h"
#include "mfma_device.h"
#include "rt.h"

namespace {

__host__ __device__ __forceinline__ int key_stride(int dim) { return (dim + 3) & ~3; }
__host__ __device__ __forceinline__ size_t head_floats(int dim, int vdim) { return (size_t)(vdim + 1) * key_stride(dim) + 4; }

__device__ __forceinline__ float log_input_gate(float raw, float b, float cap) { return cap * dm_tanh((raw + b) / cap); }
__device__ __forceinline__ float log_forget_gate(float raw, float b, float cap) {
  return dm_log_sigmoid(cap * dm_tanh((raw + b) / cap));
}

// ---- token by token -----------------------------------------------------------------------
constexpr int NT = 256, LPC = 16, COLS = NT / LPC, TB = 8;

struct StepArgs {
  const void *q, *k, *v;
  const float *gi, *gf;
  const bf16_t *bi, *bf;
  float cap, qscale;
  int T, H, dim, vdim;
  const float* st_in;
  float* slots;
  size_t slot_floats;
  int n_slots, first_slot, snapshots;
  float* o;
};

// EPL: key channels a lane holds (dim <= 16 * EPL)
template <typename A, int EPL>
__global__ __launch_bounds__(NT) void mlstm_step_kernel(StepArgs p) {
  constexpr int DP = EPL * LPC, NC = EPL / 4;
  __shared__ __attribute__((aligned(16))) float qs[TB][DP], ks[TB][DP];
  __shared__ float vs[TB][COLS], lis[TB], lfs[TB];
  const int tid = threadIdx.x, l = tid & (LPC - 1), c = tid / LPC;
  const int h = blockIdx.y, j0 = blockIdx.x * COLS, j = j0 + c;
  const int ds = key_stride(p.dim);
  const bool live = j < p.vdim, keeper = blockIdx.x == 0 && c == 0;
  const size_t head = head_floats(p.dim, p.vdim);
  const float* in = p.st_in + h * head;
  float S[EPL], n[EPL];
#pragma unroll
  for (int i = 0; i < NC; ++i) {
    const int d = 64 * i + 4 * l;
    float4 a = make_float4(0.f, 0.f, 0.f, 0.f), b = a;
    if (d < ds) {
      if (live) a = *reinterpret_cast<const float4*>(in + (size_t)j * ds + d);
      b = *reinterpret_cast<const float4*>(in + (size_t)p.vdim * ds + d);
    }
    S[4 * i] = a.x; S[4 * i + 1] = a.y; S[4 * i + 2] = a.z; S[4 * i + 3] = a.w;
    n[4 * i] = b.x; n[4 * i + 1] = b.y; n[4 * i + 2] = b.z; n[4 * i + 3] = b.w;
  }
  float m = in[(size_t)(p.vdim + 1) * ds];
  const A* q = reinterpret_cast<const A*>(p.q) + (size_t)h * p.dim;
  const A* k = reinterpret_cast<const A*>(p.k) + (size_t)h * p.dim;
  const A* v = reinterpret_cast<const A*>(p.v) + (size_t)h * p.vdim;
  for (int t0 = 0; t0 < p.T; t0 += TB) {
    const int nt = min(TB, p.T - t0);
    if (t0) __syncthreads();
    for (int i = tid; i < nt * DP; i += NT) {
      const int t = i / DP, d = i % DP;
      const size_t at = (size_t)(t0 + t) * p.H * p.dim + d;
      qs[t][d] = d < p.dim ? act_f(q[at]) * p.qscale : 0.f;
      ks[t][d] = d < p.dim ? act_f(k[at]) : 0.f;
    }
    for (int i = tid; i < nt * COLS; i += NT) {
      const int t = i / COLS, jj = j0 + i % COLS;
      vs[t][i % COLS] = jj < p.vdim ? act_f(v[(size_t)(t0 + t) * p.H * p.vdim + jj]) : 0.f;
    }
    if (tid < nt) {
      const size_t at = (size_t)(t0 + tid) * p.H + h;
      lis[tid] = log_input_gate(p.gi[at], dm_bf2f(p.bi[h]), p.cap);
      lfs[tid] = log_forget_gate(p.gf[at], dm_bf2f(p.bf[h]), p.cap);
    }
    __syncthreads();
    for (int t = 0; t < nt; ++t) {
      const float li = lis[t], f = lfs[t] + m;
      m = __builtin_fmaxf(f, li);
      const float keep = dm_exp(f - m), take = dm_exp(li - m), tv = take * vs[t][c];
      float num = 0.f, den = 0.f;
#pragma unroll
      for (int i = 0; i < NC; ++i) {
        const float4 k4 = *reinterpret_cast<const float4*>(&ks[t][64 * i + 4 * l]);
        const float4 q4 = *reinterpret_cast<const float4*>(&qs[t][64 * i + 4 * l]);
        const float kv[4] = {k4.x, k4.y, k4.z, k4.w}, qv[4] = {q4.x, q4.y, q4.z, q4.w};
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          const int x = 4 * i + e;
          S[x] = dm_fma(keep, S[x], tv * kv[e]);
          n[x] = dm_fma(keep, n[x], take * kv[e]);
          num = dm_fma(S[x], qv[e], num);
          den = dm_fma(n[x], qv[e], den);
        }
      }
      num = dm_wave_sum<16>(num);
      den = dm_wave_sum<16>(den);
      if (l == 0 && live)
        p.o[((size_t)(t0 + t) * p.H + h) * p.vdim + j] =
            num / (__builtin_fmaxf(__builtin_fabsf(den), dm_exp(-m)) + 1e-6f);
      const int tt = t0 + t;
      if (p.snapshots || tt == p.T - 1) {
        float* out = p.slots + (size_t)((p.first_slot + (p.snapshots ? tt : 0)) % p.n_slots) * p.slot_floats + h * head;
#pragma unroll
        for (int i = 0; i < NC; ++i) {
          const int d = 64 * i + 4 * l;
          if (d >= ds) continue;
          if (live)
            *reinterpret_cast<float4*>(out + (size_t)j * ds + d) =
                make_float4(S[4 * i], S[4 * i + 1], S[4 * i + 2], S[4 * i + 3]);
          if (keeper)
            *reinterpret_cast<float4*>(out + (size_t)p.vdim * ds + d) =
                make_float4(n[4 * i], n[4 * i + 1], n[4 * i + 2], n[4 * i + 3]);
        }
        if (keeper && l == 0) out[(size_t)(p.vdim + 1) * ds] = m;
      }
    }
  }
}

template <typename A>
int launch_step(ornith_ctx* ctx, const StepArgs& p) {
  const dim3 grid((p.vdim + COLS - 1) / COLS, p.H);
  if (p.dim <= 64)
    hipLaunchKernelGGL((mlstm_step_kernel<A, 4>), grid, dim3(NT), 0, ctx->stream, p);
  else if (p.dim <= 128)
    hipLaunchKernelGGL((mlstm_step_kernel<A, 8>), grid, dim3(NT), 0, ctx->stream, p);
  else if (p.dim <= 256)
    hipLaunchKernelGGL((mlstm_step_kernel<A, 16>), grid, dim3(NT), 0, ctx->stream, p);
  else
    hipLaunchKernelGGL((mlstm_step_kernel<A, 32>), grid, dim3(NT), 0, ctx->stream, p);
  ORN_LAUNCH_CHECK("mlstm_step_kernel");
  return ORNITH_OK;
}

// ---- in chunks ------------------------------------------------------------------------------
constexpr int C = 64;             // tokens a chunk
constexpr int kMaxChunks = 128;   // 8192 rows
constexpr int TILE = 64;          // key and value channels of a scan workgroup
constexpr int LS = C + 8;         // LDS row of 64 tokens, padded

typedef __bf16 m_bf16x8 __attribute__((ext_vector_type(8)));
typedef float m_f32x4 __attribute__((ext_vector_type(4)));
typedef float m_f32x16 __attribute__((ext_vector_type(16)));
typedef uint32_t m_u32x4 __attribute__((ext_vector_type(4)));

// per head and token (padded to whole chunks)
struct GateRows {
  float *r;     // F_t - m_t
  float *a;     // i_t - F_t
  float *e;     // e^(F_t + m_0 - m_t)
  float *floor_; // e^(-m_t)
  float *w;     // e^(F_C - F_t + i_t - m_C)
  float *decay; // per head and chunk: e^(F_C + m_0 - m_C)
};

__device__ __forceinline__ float scan_sum64(float v, int lane) {
#pragma unroll
  for (int s = 1; s < 64; s <<= 1) {
    const float o = __shfl_up(v, s);
    if (lane >= s) v = o + v;
  }
  return v;
}
__device__ __forceinline__ float scan_max64(float v, int lane) {
#pragma unroll
  for (int s = 1; s < 64; s <<= 1) {
    const float o = __shfl_up(v, s);
    if (lane >= s) v = __builtin_fmaxf(o, v);
  }
  return v;
}

// one workgroup a head; a wavefront a chunk, the chunks' maxima joined by one thread
__global__ __launch_bounds__(1024) void mlstm_gates_kernel(const float* gi, const float* gf, const bf16_t* bi, const bf16_t* bf,
                                                           float cap, int T, int H, int chunks, const float* st_in,
                                                           size_t head, float* st_out, GateRows g) {
  __shared__ float tot[kMaxChunks], top[kMaxChunks], m0s[kMaxChunks + 1];
  const int h = blockIdx.x, lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const float bias_i = dm_bf2f(bi[h]), bias_f = dm_bf2f(bf[h]);
  const size_t base = (size_t)h * chunks * C;
  for (int c = wave; c < chunks; c += 16) {
    const int t = c * C + lane;
    float li = -DM_INF, f = 0.f;
    if (t < T) {
      li = log_input_gate(gi[(size_t)t * H + h], bias_i, cap);
      f = log_forget_gate(gf[(size_t)t * H + h], bias_f, cap);
    }
    const float F = scan_sum64(f, lane), a = li - F, amax = scan_max64(a, lane);
    g.r[base + t] = F;  // for now
    g.a[base + t] = a;
    g.e[base + t] = amax;
    if (lane == 63) {
      tot[c] = F;
      top[c] = amax;
    }
  }
  __syncthreads();
  if (threadIdx.x == 0) {
    float m = st_in[h * head + head - 4];
    for (int c = 0; c < chunks; ++c) {
      m0s[c] = m;
      m = tot[c] + __builtin_fmaxf(m, top[c]);
    }
    m0s[chunks] = m;
    st_out[h * head + head - 4] = m;
  }
  __syncthreads();
  for (int c = wave; c < chunks; c += 16) {
    const size_t at = base + c * C + lane;
    const float F = g.r[at], a = g.a[at], m0 = m0s[c], top_t = __builtin_fmaxf(m0, g.e[at]);
    // m_t = F + top_t, so F_t - m_t = -top_t
    g.r[at] = -top_t;
    g.e[at] = dm_exp(m0 - top_t);
    g.floor_[at] = dm_exp(-(F + top_t));
    const float top_c = __builtin_fmaxf(m0, top[c]);
    g.w[at] = dm_exp(a - top_c);
    if (lane == 0) g.decay[(size_t)h * chunks + c] = dm_exp(m0 - top_c);
  }
}

// S_0 of a chunk lies in the matrix cores' order (s0_at), bf16 high parts, then low parts.
struct ScanArgs {
  const bf16_t *k, *v;
  const float *w, *decay;
  int T, H, dim, vdim, DP, VP, chunks, c0, c1;  // chunks [c0, c1) of the call
  const float* st_in;
  float* st_out;
  bf16_t *s_hi, *s_lo;  // [H][c1 - c0][VP][DP]
  float* n0;            // [H][c1 - c0][DP]
};

// One workgroup walks a 64 x 64 (key x value) tile of one head's state through the chunks. Both
// operands of the outer products run over tokens, so keys and values are turned in LDS: a thread brings
// two tokens of eight channels and writes eight token pairs. The next chunk's loads are in flight
// meanwhile.
__global__ __launch_bounds__(256) void mlstm_scan_kernel(ScanArgs p) {
  __shared__ __attribute__((aligned(16))) bf16_t Khi[TILE][LS], Klo[TILE][LS], Vt[TILE][LS];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, l32 = lane & 31, lh = lane >> 5;
  const int h = blockIdx.z, d0 = blockIdx.x * TILE, j0 = blockIdx.y * TILE;
  const int wd = (wave & 1) * 32, wj = (wave >> 1) * 32;
  const int ds = key_stride(p.dim);
  const size_t head = head_floats(p.dim, p.vdim);
  const float* in = p.st_in + h * head;
  float* out = p.st_out + h * head;
  const bool norm_tile = blockIdx.y == 0 && wj == 0;
  // acc element 4q + e: S[value j][key d + e]
  const int j = j0 + wj + l32;
  m_f32x16 acc, accn;
#pragma unroll
  for (int q = 0; q < 4; ++q) {
    const int d = d0 + wd + 8 * q + 4 * lh;
    float4 s = make_float4(0.f, 0.f, 0.f, 0.f), n = s;
    if (d < ds) {
      if (j < p.vdim) s = *reinterpret_cast<const float4*>(in + (size_t)j * ds + d);
      if (norm_tile) n = *reinterpret_cast<const float4*>(in + (size_t)p.vdim * ds + d);
    }
    acc[4 * q] = s.x; acc[4 * q + 1] = s.y; acc[4 * q + 2] = s.z; acc[4 * q + 3] = s.w;
    accn[4 * q] = n.x; accn[4 * q + 1] = n.y; accn[4 * q + 2] = n.z; accn[4 * q + 3] = n.w;
  }
  m_bf16x8 ones;
#pragma unroll
  for (int i = 0; i < 8; ++i) ones[i] = (__bf16)1.0f;

  // eight channels, two tokens: four neighbouring lanes read 64 bytes of a row, and the sixteen token
  // pairs of a wavefront keep its LDS writes two to a bank
  const int oct = (tid & 3) + 4 * (tid >> 7), pair = (tid >> 2) & 31;
  const bool kin = d0 + 8 * oct < p.dim, vin = j0 + 8 * oct < p.vdim;
  const bf16_t* kp = p.k + (size_t)h * p.dim + d0 + 8 * oct;
  const bf16_t* vp = p.v + (size_t)h * p.vdim + j0 + 8 * oct;
  const size_t krow = (size_t)p.H * p.dim, vrow = (size_t)p.H * p.vdim;
  const float* wrow = p.w + (size_t)h * p.chunks * C;
  m_u32x4 kr[2], vr[2];
  float wt[2];
  auto load = [&](int c) {
    const m_u32x4 zero = {0, 0, 0, 0};
#pragma unroll
    for (int i = 0; i < 2; ++i) {
      const int t = c * C + 2 * pair + i, tc = min(t, p.T - 1);
      kr[i] = kin ? *reinterpret_cast<const m_u32x4*>(kp + (size_t)tc * krow) : zero;
      vr[i] = vin ? *reinterpret_cast<const m_u32x4*>(vp + (size_t)tc * vrow) : zero;
      wt[i] = wrow[t];  // zero past the last token
    }
  };
  load(p.c0);
  float decay = p.decay[(size_t)h * p.chunks + p.c0];
  for (int c = p.c0; c < p.c1; ++c) {
    // this chunk's S_0
    const size_t cb = ((size_t)h * (p.c1 - p.c0) + (c - p.c0)) * p.VP * p.DP;
#pragma unroll
    for (int q = 0; q < 4; ++q) {
      const int d = d0 + wd + 8 * q + 4 * lh;
      uint2 hi, lo;
      split2(acc[4 * q], acc[4 * q + 1], hi.x, lo.x);
      split2(acc[4 * q + 2], acc[4 * q + 3], hi.y, lo.y);
      if (d < p.DP) {
        const size_t at = cb + s0_at(p.DP, j, d);
        *reinterpret_cast<uint2*>(p.s_hi + at) = hi;
        *reinterpret_cast<uint2*>(p.s_lo + at) = lo;
        if (norm_tile && l32 == 0)
          *reinterpret_cast<float4*>(p.n0 + ((size_t)h * (p.c1 - p.c0) + (c - p.c0)) * p.DP + d) =
              make_float4(accn[4 * q], accn[4 * q + 1], accn[4 * q + 2], accn[4 * q + 3]);
      }
    }
    // turn the chunk: word [channel][token pair]
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const float k0[2] = {dm_bf2f_lo(kr[0][i]), dm_bf2f_hi(kr[0][i])}, k1[2] = {dm_bf2f_lo(kr[1][i]), dm_bf2f_hi(kr[1][i])};
#pragma unroll
      for (int b = 0; b < 2; ++b) {
        uint32_t hi, lo;
        split2(k0[b] * wt[0], k1[b] * wt[1], hi, lo);
        const int ch = 8 * oct + 2 * i + b;
        *reinterpret_cast<uint32_t*>(&Khi[ch][2 * pair]) = hi;
        *reinterpret_cast<uint32_t*>(&Klo[ch][2 * pair]) = lo;
        *reinterpret_cast<uint32_t*>(&Vt[ch][2 * pair]) =
            b ? (vr[0][i] >> 16) | (vr[1][i] & 0xffff0000u) : (vr[0][i] & 0xffffu) | (vr[1][i] << 16);
      }
    }
    const float dec = decay;
    if (c + 1 < p.c1) {
      load(c + 1);
      decay = p.decay[(size_t)h * p.chunks + c + 1];
    }
    __syncthreads();
#pragma unroll
    for (int i = 0; i < 16; ++i) acc[i] *= dec;
    if (norm_tile) {
#pragma unroll
      for (int i = 0; i < 16; ++i) accn[i] *= dec;
    }
#pragma unroll
    for (int kk = 0; kk < 4; ++kk) {
      const m_bf16x8 ah = *reinterpret_cast<const m_bf16x8*>(&Khi[wd + l32][16 * kk + 8 * lh]);
      const m_bf16x8 al = *reinterpret_cast<const m_bf16x8*>(&Klo[wd + l32][16 * kk + 8 * lh]);
      const m_bf16x8 bv = *reinterpret_cast<const m_bf16x8*>(&Vt[wj + l32][16 * kk + 8 * lh]);
      acc = __builtin_amdgcn_mfma_f32_32x32x16_bf16(ah, bv, acc, 0, 0, 0);
      acc = __builtin_amdgcn_mfma_f32_32x32x16_bf16(al, bv, acc, 0, 0, 0);
      if (norm_tile) {
        accn = __builtin_amdgcn_mfma_f32_32x32x16_bf16(ah, ones, accn, 0, 0, 0);
        accn = __builtin_amdgcn_mfma_f32_32x32x16_bf16(al, ones, accn, 0, 0, 0);
      }
    }
    __syncthreads();
  }
#pragma unroll
  for (int q = 0; q < 4; ++q) {
    const int d = d0 + wd + 8 * q + 4 * lh;
    if (d >= ds) continue;
    if (j < p.vdim)
      *reinterpret_cast<float4*>(out + (size_t)j * ds + d) = make_float4(acc[4 * q], acc[4 * q + 1], acc[4 * q + 2], acc[4 * q + 3]);
    if (norm_tile && l32 == 0)
      *reinterpret_cast<float4*>(out + (size_t)p.vdim * ds + d) = make_float4(accn[4 * q], accn[4 * q + 1], accn[4 * q + 2], accn[4 * q + 3]);
  }
}

struct OutArgs {
  const bf16_t *q, *k, *v;
  GateRows g;
  float qscale;
  int T, H, dim, vdim, VP, chunks, c0, c1;
  const bf16_t *s_hi, *s_lo;
  const float* n0;
  float* o;
};

// One workgroup: one chunk of one head, 32 * NV value channels. Wavefront (wq, wv) makes the outputs of
// 32 queries (two groups of sixteen) for half the channels. All products run transposed, so that a lane
// owns a query from the scores to the output: O^T = S_0 Q^T, then + V^T P^T.
template <int KD, int NV>
__global__ __launch_bounds__(256) void mlstm_out_kernel(OutArgs p) {
  constexpr int DP = KD * 32, VB = 32 * NV;
  __shared__ __attribute__((aligned(16))) bf16_t Vt[VB][LS];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, l16 = lane & 15, lg = lane >> 4;
  const int c = p.c0 + blockIdx.x, h = blockIdx.z, jb = blockIdx.y * VB;
  const int wq = (wave & 1) * 32, wv = (wave >> 1) * (VB / 2);
  const int t0 = c * C;
  // values, turned: a thread brings two tokens of eight channels
  for (int i = tid; i < (VB / 8) * (C / 2); i += 256) {
    const int oct = (i & 3) + 4 * (i >> 7), pair = (i >> 2) & 31;  // as in the scan
    const m_u32x4 zero = {0, 0, 0, 0};
    m_u32x4 a = zero, b = zero;
    if (jb + 8 * oct < p.vdim) {
      const bf16_t* src = p.v + (size_t)h * p.vdim + jb + 8 * oct;
      a = *reinterpret_cast<const m_u32x4*>(src + (size_t)min(t0 + 2 * pair, p.T - 1) * p.H * p.vdim);
      b = *reinterpret_cast<const m_u32x4*>(src + (size_t)min(t0 + 2 * pair + 1, p.T - 1) * p.H * p.vdim);
    }
    const int at = (2 * pair & 32) + vt_pos(2 * pair & 31);
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      *reinterpret_cast<uint32_t*>(&Vt[8 * oct + 2 * e][at]) = (a[e] & 0xffffu) | (b[e] << 16);
      *reinterpret_cast<uint32_t*>(&Vt[8 * oct + 2 * e + 1][at]) = (a[e] >> 16) | (b[e] & 0xffff0000u);
    }
  }
  const size_t gb = (size_t)h * p.chunks * C + t0;
  // queries: fragment kk holds channels 32 kk + 8 lg .. of query l16
  m_bf16x8 qf[2][KD];
  int tq[2];
  float er[2], rr[2], fl[2];
#pragma unroll
  for (int s = 0; s < 2; ++s) {
    const int ql = wq + 16 * s + l16;
    tq[s] = t0 + ql;
    er[s] = p.g.e[gb + ql];
    rr[s] = p.g.r[gb + ql];
    fl[s] = p.g.floor_[gb + ql];
    const bf16_t* src = p.q + ((size_t)min(tq[s], p.T - 1) * p.H + h) * p.dim;
#pragma unroll
    for (int kk = 0; kk < KD; ++kk) {
      const int d = 32 * kk + 8 * lg;
      m_u32x4 x = {0, 0, 0, 0};
      if (d < p.dim) x = *reinterpret_cast<const m_u32x4*>(src + d);
      qf[s][kk] = __builtin_bit_cast(m_bf16x8, x);
    }
  }
  // the part of S_0
  const size_t cb = (size_t)h * (p.c1 - p.c0) + blockIdx.x;
  const bf16_t* sh = p.s_hi + cb * p.VP * DP;
  const bf16_t* sl = p.s_lo + cb * p.VP * DP;
  m_f32x4 acc[2][NV];
#pragma unroll
  for (int s = 0; s < 2; ++s)
#pragma unroll
    for (int vt = 0; vt < NV; ++vt) acc[s][vt] = m_f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int vt = 0; vt < NV; ++vt) {
    const size_t row = (size_t)((jb + wv) / 16 + vt) * KD * 512 + (size_t)lane * 8;
#pragma unroll
    for (int kk = 0; kk < KD; ++kk) {
      const m_bf16x8 ah = *reinterpret_cast<const m_bf16x8*>(sh + row + kk * 512);
      const m_bf16x8 al = *reinterpret_cast<const m_bf16x8*>(sl + row + kk * 512);
#pragma unroll
      for (int s = 0; s < 2; ++s) {
        acc[s][vt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(ah, qf[s][kk], acc[s][vt], 0, 0, 0);
        acc[s][vt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(al, qf[s][kk], acc[s][vt], 0, 0, 0);
      }
    }
  }
  float den[2] = {0.f, 0.f};
  const float* n0 = p.n0 + cb * DP;
#pragma unroll
  for (int kk = 0; kk < KD; ++kk)
#pragma unroll
    for (int e = 0; e < 8; ++e) {
      const float nv = n0[32 * kk + 8 * lg + e];
#pragma unroll
      for (int s = 0; s < 2; ++s) den[s] = dm_fma(nv, (float)qf[s][kk][e], den[s]);
    }
#pragma unroll
  for (int s = 0; s < 2; ++s) {
    const float x = er[s] * p.qscale;
    den[s] *= x;
#pragma unroll
    for (int vt = 0; vt < NV; ++vt) acc[s][vt] *= x;
  }
  __syncthreads();
  // the chunk's own tokens, 32 at a time (none after this wavefront's last query)
#pragma unroll
  for (int half = 0; half < 2; ++half) {
    if (32 * half > wq + 31) break;
    m_f32x4 sc[2][2];
#pragma unroll
    for (int kt = 0; kt < 2; ++kt) {
#pragma unroll
      for (int s = 0; s < 2; ++s) sc[s][kt] = m_f32x4{0.f, 0.f, 0.f, 0.f};
      const bf16_t* src = p.k + ((size_t)min(t0 + 32 * half + 16 * kt + l16, p.T - 1) * p.H + h) * p.dim;
#pragma unroll
      for (int kk = 0; kk < KD; ++kk) {
        const int d = 32 * kk + 8 * lg;
        m_u32x4 x = {0, 0, 0, 0};
        if (d < p.dim) x = *reinterpret_cast<const m_u32x4*>(src + d);
        const m_bf16x8 kf = __builtin_bit_cast(m_bf16x8, x);
#pragma unroll
        for (int s = 0; s < 2; ++s) sc[s][kt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf, qf[s][kk], sc[s][kt], 0, 0, 0);
      }
    }
    // P: key 32 half + 16 kt + 4 lg + r of query tq
    m_bf16x8 ph[2], pl[2];
#pragma unroll
    for (int s = 0; s < 2; ++s) {
      uint32_t hi[4], lo[4];
#pragma unroll
      for (int kt = 0; kt < 2; ++kt) {
        float w[4];
        const float4 a4 = *reinterpret_cast<const float4*>(p.g.a + gb + 32 * half + 16 * kt + 4 * lg);
        const float av[4] = {a4.x, a4.y, a4.z, a4.w};
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int key = 32 * half + 16 * kt + 4 * lg + r;
          const bool see = key <= wq + 16 * s + l16;
          w[r] = see ? dm_exp2_hw((rr[s] + av[r]) * 1.44269504088896341f) * (sc[s][kt][r] * p.qscale) : 0.f;
        }
        split2(w[0], w[1], hi[2 * kt], lo[2 * kt]);
        split2(w[2], w[3], hi[2 * kt + 1], lo[2 * kt + 1]);
        // the sum over tokens, in the lanes that share a query
        float ws = (w[0] + w[1]) + (w[2] + w[3]);
        den[s] += ws;
      }
      const m_u32x4 hv = {hi[0], hi[1], hi[2], hi[3]}, lv = {lo[0], lo[1], lo[2], lo[3]};
      ph[s] = __builtin_bit_cast(m_bf16x8, hv);
      pl[s] = __builtin_bit_cast(m_bf16x8, lv);
    }
#pragma unroll
    for (int vt = 0; vt < NV; ++vt) {
      const m_bf16x8 vf = *reinterpret_cast<const m_bf16x8*>(&Vt[wv + 16 * vt + l16][32 * half + 8 * lg]);
#pragma unroll
      for (int s = 0; s < 2; ++s) {
        acc[s][vt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf, ph[s], acc[s][vt], 0, 0, 0);
        acc[s][vt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf, pl[s], acc[s][vt], 0, 0, 0);
      }
    }
  }
#pragma unroll
  for (int s = 0; s < 2; ++s) {
    const float d = dm_sum_groups16(den[s]);
    const float inv = 1.0f / (__builtin_fmaxf(__builtin_fabsf(d), fl[s]) + 1e-6f);
    if (tq[s] >= p.T) continue;
    float* dst = p.o + ((size_t)tq[s] * p.H + h) * p.vdim;
#pragma unroll
    for (int vt = 0; vt < NV; ++vt) {
      const int jj = jb + wv + 16 * vt + 4 * lg;
      if (jj < p.vdim)
        *reinterpret_cast<float4*>(dst + jj) = make_float4(acc[s][vt][0] * inv, acc[s][vt][1] * inv, acc[s][vt][2] * inv, acc[s][vt][3] * inv);
    }
  }
}

template <int KD>
void launch_out(ornith_ctx* ctx, const OutArgs& p) {
  if (p.vdim <= 64)
    hipLaunchKernelGGL((mlstm_out_kernel<KD, 2>), dim3(p.c1 - p.c0, 1, p.H), dim3(256), 0, ctx->stream, p);
  else
    hipLaunchKernelGGL((mlstm_out_kernel<KD, 4>), dim3(p.c1 - p.c0, p.VP / 128, p.H), dim3(256), 0, ctx->stream, p);
}

int run_chunked(ornith_ctx* ctx, const ornith_mlstm_call* c, float* st_out) {
  const int KD = c->dim <= 64 ? 2 : c->dim <= 128 ? 4 : 8, DP = KD * 32;
  const int VP = c->vdim <= 64 ? 64 : (c->vdim + 127) / 128 * 128;
  const int chunks = (c->T + C - 1) / C;
  const size_t head = head_floats(c->dim, c->vdim);
  // chunks a scan / output launch pair takes: what the scan writes (and the outputs read) should
  // still be in the last-level cache
  const size_t per_chunk = (size_t)c->H * VP * DP * 4;
  int block = (int)((size_t(96) << 20) / per_chunk);
  block = block < 8 ? 8 : block > chunks ? chunks : block;
  const size_t rows = (size_t)c->H * chunks * C;
  void* base = nullptr;
  int rc = ornith_scratch(ctx, 5 * rows * 4 + (size_t)c->H * chunks * 4 + (size_t)c->H * block * DP * 4 + per_chunk * block + 16 * 256, &base);
  if (rc) return rc;
  ScratchCursor sc(base);
  GateRows g;
  g.r = sc.take<float>(rows);
  g.a = sc.take<float>(rows);
  g.e = sc.take<float>(rows);
  g.floor_ = sc.take<float>(rows);
  g.w = sc.take<float>(rows);
  g.decay = sc.take<float>((size_t)c->H * chunks);
  float* n0 = sc.take<float>((size_t)c->H * block * DP);
  bf16_t* s_hi = sc.take<bf16_t>((size_t)c->H * block * VP * DP);
  bf16_t* s_lo = sc.take<bf16_t>((size_t)c->H * block * VP * DP);
  hipLaunchKernelGGL(mlstm_gates_kernel, dim3(c->H), dim3(1024), 0, ctx->stream, c->d_gi, c->d_gf, (const bf16_t*)c->d_bi,
                     (const bf16_t*)c->d_bf, c->gate_cap, c->T, c->H, chunks, c->d_state_in, head, st_out, g);
  ORN_LAUNCH_CHECK("mlstm_gates_kernel");
  for (int c0 = 0; c0 < chunks; c0 += block) {
    const int c1 = c0 + block < chunks ? c0 + block : chunks;
    ScanArgs s{(const bf16_t*)c->d_k, (const bf16_t*)c->d_v, g.w, g.decay, c->T, c->H, c->dim, c->vdim, DP, VP, chunks, c0, c1,
               c0 ? st_out : c->d_state_in, st_out, s_hi, s_lo, n0};
    hipLaunchKernelGGL(mlstm_scan_kernel, dim3(DP / TILE, VP / TILE, c->H), dim3(256), 0, ctx->stream, s);
    ORN_LAUNCH_CHECK("mlstm_scan_kernel");
    OutArgs o{(const bf16_t*)c->d_q, (const bf16_t*)c->d_k, (const bf16_t*)c->d_v, g, 1.0f / __builtin_sqrtf((float)c->dim),
              c->T, c->H, c->dim, c->vdim, VP, chunks, c0, c1, s_hi, s_lo, n0, c->d_o};
    if (KD == 2) launch_out<2>(ctx, o);
    else if (KD == 4) launch_out<4>(ctx, o);
    else launch_out<8>(ctx, o);
    ORN_LAUNCH_CHECK("mlstm_out_kernel");
  }
  return ORNITH_OK;
}

}  // namespace

extern "C" {

size_t ornith_mlstm_state_floats(int H, int dim, int vdim) { return (size_t)H * head_floats(dim, vdim); }

int ornith_mlstm(ornith_ctx* ctx, const ornith_mlstm_call* c) {
  ORN_REQUIRE(ctx && c && c->d_q && c->d_k && c->d_v && c->d_gi && c->d_gf && c->d_bi && c->d_bf && c->d_state_in &&
                  c->d_slots && c->d_o, "mlstm: null argument");
  ORN_REQUIRE(c->T >= 1 && c->H >= 1 && c->H <= 65535 && c->dim >= 1 && c->dim <= 512 && c->vdim >= 1 && c->gate_cap > 0,
              "mlstm: T=%d H=%d dim=%d (at most 512) vdim=%d cap=%g", c->T, c->H, c->dim, c->vdim, c->gate_cap);
  ORN_REQUIRE(c->n_slots >= 1 && c->first_slot >= 0 && c->first_slot < c->n_slots && (!c->snapshots || c->T < c->n_slots),
              "mlstm: slot %d of %d for %d rows", c->first_slot, c->n_slots, c->T);
  const size_t slot = ornith_mlstm_state_floats(c->H, c->dim, c->vdim);
  float* first = c->d_slots + (size_t)c->first_slot * slot;
  ORN_REQUIRE(first != c->d_state_in, "mlstm: the slot a call starts from is not one it may write");
  if (c->act == ORNITH_BF16 && c->T >= C && c->T <= kMaxChunks * C && !c->snapshots && ornith_option_mlstm_chunked() &&
      c->dim % 8 == 0 && c->vdim % 8 == 0 && c->dim <= 256)
    return run_chunked(ctx, c, first);
  StepArgs p{c->d_q, c->d_k, c->d_v, c->d_gi, c->d_gf, (const bf16_t*)c->d_bi, (const bf16_t*)c->d_bf, c->gate_cap,
             1.0f / __builtin_sqrtf((float)c->dim), c->T, c->H, c->dim, c->vdim, c->d_state_in, c->d_slots, slot, c->n_slots,
             c->first_slot, c->snapshots, c->d_o};
  return c->act == ORNITH_F32 ? launch_step<float>(ctx, p) : launch_step<bf16_t>(ctx, p);
}

}  // extern "C"
