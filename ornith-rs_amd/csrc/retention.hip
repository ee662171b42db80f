// Retention: a matrix state a head, S (value x key channels), that fades by the head's fixed decay (Sun et
// al., "Retentive Network"), with rotary positions on queries and keys. The arithmetic is stated at
// ornith_retention in ornith_hip.h. The state of a head in memory, fp32: S [vdim][ds], ds = dim rounded up
// to 4 (the padding stays zero).
//
// Token by token (decode widths, 32-bit models): a workgroup takes sixteen value channels of one head,
// sixteen lanes a channel, the state in registers across the call's tokens; it turns the queries and keys
// it stages itself.
//
// In chunks of 64 tokens (prefill widths, bf16), three launches. With S_0 what a chunk of n tokens starts
// from and g the decay,
//   o_t = g^(t+1) S_0 q_t + sum_{s<=t} g^(t-s) (q_t . k_s) v_s,   S_n = g^n S_0 + sum_s g^(n-1-s) v_s k_s^T
// (every power is at most the first): retention_turn_kernel turns and scales queries and keys;
// retention_scan_kernel walks S from chunk to chunk, tile by tile independent, leaving each chunk's S_0;
// retention_out_kernel makes the outputs, all chunks at once. v are bf16 numbers; turned q and k, S_0, the
// weights and the weighted keys go to the matrix cores as two bf16 parts each, so nothing of the
// recurrence is rounded to bf16.
#include <cmath>
#include <vector>

#include "act_device.h"
#include "mfma_device.h"
#include "rt.h"

namespace {

__host__ __device__ __forceinline__ int key_stride(int dim) { return (dim + 3) & ~3; }
__host__ __device__ __forceinline__ size_t head_floats(int dim, int vdim) { return (size_t)vdim * key_stride(dim); }

struct RotArgs {
  const float *cos_t, *sin_t;
  int half, offset;  // dimension i < half pairs with i + half
};

// element d of a row at position pos, turned
template <typename A>
__device__ __forceinline__ float turned(const A* row, int d, int pos, const RotArgs& r) {
  const float x = act_f(row[d]);
  if (d >= 2 * r.half) return x;
  const bool second = d >= r.half;
  const int i = second ? d - r.half : d;
  const float y = act_f(row[second ? i : d + r.half]);
  const size_t at = (size_t)pos * r.half + i;
  const float c = r.cos_t[at], s = r.sin_t[at];
  return second ? dm_fma(y, s, x * c) : dm_fma(-y, s, x * c);
}

// ---- token by token -----------------------------------------------------------------------
constexpr int NT = 256, LPC = 16, COLS = NT / LPC, TB = 8;

struct StepArgs {
  const void *q, *k, *v;
  RotArgs rot;
  const float* decay;
  float kscale;
  int T, H, dim, vdim;
  const float* st_in;
  float* slots;
  size_t slot_floats;
  int n_slots, first_slot, snapshots;
  float* o;
};

// EPL: key channels a lane holds (dim <= 16 * EPL)
template <typename A, int EPL>
__global__ __launch_bounds__(NT) void retention_step_kernel(StepArgs p) {
  constexpr int DP = EPL * LPC, NC = EPL / 4;
  __shared__ __attribute__((aligned(16))) float qs[TB][DP], ks[TB][DP];
  __shared__ float vs[TB][COLS];
  const int tid = threadIdx.x, l = tid & (LPC - 1), c = tid / LPC;
  const int h = blockIdx.y, j0 = blockIdx.x * COLS, j = j0 + c;
  const int ds = key_stride(p.dim);
  const bool live = j < p.vdim;
  const size_t head = head_floats(p.dim, p.vdim);
  const float* in = p.st_in + h * head;
  float S[EPL];
#pragma unroll
  for (int i = 0; i < NC; ++i) {
    const int d = 64 * i + 4 * l;
    float4 a = make_float4(0.f, 0.f, 0.f, 0.f);
    if (d < ds && live) a = *reinterpret_cast<const float4*>(in + (size_t)j * ds + d);
    S[4 * i] = a.x; S[4 * i + 1] = a.y; S[4 * i + 2] = a.z; S[4 * i + 3] = a.w;
  }
  const float g = p.decay[(size_t)h * ORNITH_DECAY_POWERS + 1];
  const A* q = reinterpret_cast<const A*>(p.q) + (size_t)h * p.dim;
  const A* k = reinterpret_cast<const A*>(p.k) + (size_t)h * p.dim;
  const A* v = reinterpret_cast<const A*>(p.v) + (size_t)h * p.vdim;
  for (int t0 = 0; t0 < p.T; t0 += TB) {
    const int nt = min(TB, p.T - t0);
    if (t0) __syncthreads();
    for (int i = tid; i < nt * DP; i += NT) {
      const int t = i / DP, d = i % DP, pos = p.rot.offset + t0 + t;
      const size_t row = (size_t)(t0 + t) * p.H * p.dim;
      qs[t][d] = d < p.dim ? turned(q + row, d, pos, p.rot) : 0.f;
      ks[t][d] = d < p.dim ? turned(k + row, d, pos, p.rot) * p.kscale : 0.f;
    }
    for (int i = tid; i < nt * COLS; i += NT) {
      const int t = i / COLS, jj = j0 + i % COLS;
      vs[t][i % COLS] = jj < p.vdim ? act_f(v[(size_t)(t0 + t) * p.H * p.vdim + jj]) : 0.f;
    }
    __syncthreads();
    for (int t = 0; t < nt; ++t) {
      const float tv = vs[t][c];
      float num = 0.f;
#pragma unroll
      for (int i = 0; i < NC; ++i) {
        const float4 k4 = *reinterpret_cast<const float4*>(&ks[t][64 * i + 4 * l]);
        const float4 q4 = *reinterpret_cast<const float4*>(&qs[t][64 * i + 4 * l]);
        const float kv[4] = {k4.x, k4.y, k4.z, k4.w}, qv[4] = {q4.x, q4.y, q4.z, q4.w};
#pragma unroll
        for (int e = 0; e < 4; ++e) {
          const int x = 4 * i + e;
          S[x] = dm_fma(g, S[x], tv * kv[e]);
          num = dm_fma(S[x], qv[e], num);
        }
      }
      num = dm_wave_sum<16>(num);
      const int tt = t0 + t;
      if (l == 0 && live) p.o[((size_t)tt * p.H + h) * p.vdim + j] = num;
      if (live && (p.snapshots || tt == p.T - 1)) {
        float* out = p.slots + (size_t)((p.first_slot + (p.snapshots ? tt : 0)) % p.n_slots) * p.slot_floats + h * head;
#pragma unroll
        for (int i = 0; i < NC; ++i) {
          const int d = 64 * i + 4 * l;
          if (d < ds)
            *reinterpret_cast<float4*>(out + (size_t)j * ds + d) = make_float4(S[4 * i], S[4 * i + 1], S[4 * i + 2], S[4 * i + 3]);
        }
      }
    }
  }
}

template <typename A>
int launch_step(ornith_ctx* ctx, const StepArgs& p) {
  const dim3 grid((p.vdim + COLS - 1) / COLS, p.H);
  if (p.dim <= 64)
    hipLaunchKernelGGL((retention_step_kernel<A, 4>), grid, dim3(NT), 0, ctx->stream, p);
  else if (p.dim <= 128)
    hipLaunchKernelGGL((retention_step_kernel<A, 8>), grid, dim3(NT), 0, ctx->stream, p);
  else if (p.dim <= 256)
    hipLaunchKernelGGL((retention_step_kernel<A, 16>), grid, dim3(NT), 0, ctx->stream, p);
  else
    hipLaunchKernelGGL((retention_step_kernel<A, 32>), grid, dim3(NT), 0, ctx->stream, p);
  ORN_LAUNCH_CHECK("retention_step_kernel");
  return ORNITH_OK;
}

// ---- in chunks ------------------------------------------------------------------------------
constexpr int C = 64;     // tokens a chunk
constexpr int TILE = 64;  // key and value channels of a scan workgroup
constexpr int LS = C + 8; // LDS row of 64 tokens, padded

typedef __bf16 r_bf16x8 __attribute__((ext_vector_type(8)));
typedef float r_f32x4 __attribute__((ext_vector_type(4)));
typedef float r_f32x16 __attribute__((ext_vector_type(16)));
typedef uint32_t r_u32x4 __attribute__((ext_vector_type(4)));

// [T][H*dim] each
struct TurnedRows {
  bf16_t *q_hi, *q_lo, *k_hi, *k_lo;
};

// one workgroup a token; a thread turns four channels (dim is a multiple of 8)
__global__ __launch_bounds__(NT) void retention_turn_kernel(const bf16_t* q, const bf16_t* k, RotArgs r, float kscale, int H,
                                                            int dim, TurnedRows out) {
  const int t = blockIdx.x, pos = r.offset + t, n4 = H * dim / 4;
  const size_t base = (size_t)t * H * dim;
  const bool vec = r.half % 4 == 0;
  for (int i = threadIdx.x; i < 2 * n4; i += NT) {
    const bool is_k = i >= n4;
    const int e0 = 4 * (is_k ? i - n4 : i), d = e0 % dim;
    const bf16_t* row = (is_k ? k : q) + base + (e0 - d);
    float v[4];
    if (vec && d < 2 * r.half) {
      const bool second = d >= r.half;
      const int i0 = second ? d - r.half : d;
      float x[4], y[4];
      act_load<4>(row + d, x);
      act_load<4>(row + (second ? i0 : d + r.half), y);
      const size_t at = (size_t)pos * r.half + i0;
      const float4 c4 = *reinterpret_cast<const float4*>(r.cos_t + at), s4 = *reinterpret_cast<const float4*>(r.sin_t + at);
      const float c[4] = {c4.x, c4.y, c4.z, c4.w}, s[4] = {s4.x, s4.y, s4.z, s4.w};
#pragma unroll
      for (int e = 0; e < 4; ++e) v[e] = second ? dm_fma(y[e], s[e], x[e] * c[e]) : dm_fma(-y[e], s[e], x[e] * c[e]);
    } else {
#pragma unroll
      for (int e = 0; e < 4; ++e) v[e] = turned(row, d + e, pos, r);
    }
    if (is_k) {
#pragma unroll
      for (int e = 0; e < 4; ++e) v[e] *= kscale;
    }
    uint2 hi, lo;
    split2(v[0], v[1], hi.x, lo.x);
    split2(v[2], v[3], hi.y, lo.y);
    *reinterpret_cast<uint2*>((is_k ? out.k_hi : out.q_hi) + base + e0) = hi;
    *reinterpret_cast<uint2*>((is_k ? out.k_lo : out.q_lo) + base + e0) = lo;
  }
}

struct ScanArgs {
  const bf16_t *k_hi, *k_lo, *v;
  const float* decay;
  int T, H, dim, vdim, DP, VP, c0, c1;  // chunks [c0, c1) of the call
  const float* st_in;
  float* st_out;
  bf16_t *s_hi, *s_lo;  // [H][c1 - c0][VP][DP]
};

// One workgroup walks a 64 x 64 (key x value) tile of one head's state through the chunks. Both
// operands of the outer products run over tokens, so keys and values are turned in LDS: a thread brings
// two tokens of eight channels and writes eight token pairs. The next chunk's loads are in flight
// meanwhile.
__global__ __launch_bounds__(256) void retention_scan_kernel(ScanArgs p) {
  __shared__ __attribute__((aligned(16))) bf16_t Khi[TILE][LS], Klo[TILE][LS], Vt[TILE][LS];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, l32 = lane & 31, lh = lane >> 5;
  const int h = blockIdx.z, d0 = blockIdx.x * TILE, j0 = blockIdx.y * TILE;
  const int wd = (wave & 1) * 32, wj = (wave >> 1) * 32;
  const int ds = key_stride(p.dim);
  const size_t head = head_floats(p.dim, p.vdim);
  const float* in = p.st_in + h * head;
  float* out = p.st_out + h * head;
  const float* pw = p.decay + (size_t)h * ORNITH_DECAY_POWERS;
  // acc element 4q + e: S[value j][key d + e]
  const int j = j0 + wj + l32;
  r_f32x16 acc;
#pragma unroll
  for (int q = 0; q < 4; ++q) {
    const int d = d0 + wd + 8 * q + 4 * lh;
    float4 s = make_float4(0.f, 0.f, 0.f, 0.f);
    if (d < ds && j < p.vdim) s = *reinterpret_cast<const float4*>(in + (size_t)j * ds + d);
    acc[4 * q] = s.x; acc[4 * q + 1] = s.y; acc[4 * q + 2] = s.z; acc[4 * q + 3] = s.w;
  }
  // eight channels, two tokens: four neighbouring lanes read 64 bytes of a row, and the sixteen token
  // pairs of a wavefront keep its LDS writes two to a bank
  const int oct = (tid & 3) + 4 * (tid >> 7), pair = (tid >> 2) & 31;
  const bool kin = d0 + 8 * oct < p.dim, vin = j0 + 8 * oct < p.vdim;
  const size_t kat = (size_t)h * p.dim + d0 + 8 * oct;
  const bf16_t* vp = p.v + (size_t)h * p.vdim + j0 + 8 * oct;
  const size_t krow = (size_t)p.H * p.dim, vrow = (size_t)p.H * p.vdim;
  r_u32x4 kh[2], kl[2], vr[2];
  auto load = [&](int c) {
    const r_u32x4 zero = {0, 0, 0, 0};
#pragma unroll
    for (int i = 0; i < 2; ++i) {
      const int t = min(c * C + 2 * pair + i, p.T - 1);
      kh[i] = kin ? *reinterpret_cast<const r_u32x4*>(p.k_hi + kat + (size_t)t * krow) : zero;
      kl[i] = kin ? *reinterpret_cast<const r_u32x4*>(p.k_lo + kat + (size_t)t * krow) : zero;
      vr[i] = vin ? *reinterpret_cast<const r_u32x4*>(vp + (size_t)t * vrow) : zero;
    }
  };
  load(p.c0);
  for (int c = p.c0; c < p.c1; ++c) {
    const int n = min(C, p.T - c * C);  // tokens of this chunk; the others' weight is zero
    float wt[2];
#pragma unroll
    for (int i = 0; i < 2; ++i) {
      const int t = 2 * pair + i;
      wt[i] = t < n ? pw[n - 1 - t] : 0.f;
    }
    const float dec = pw[n];
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
      }
    }
    // turn the chunk: word [channel][token pair]
#pragma unroll
    for (int i = 0; i < 4; ++i) {
      const float k0[2] = {dm_bf2f_lo(kh[0][i]) + dm_bf2f_lo(kl[0][i]), dm_bf2f_hi(kh[0][i]) + dm_bf2f_hi(kl[0][i])};
      const float k1[2] = {dm_bf2f_lo(kh[1][i]) + dm_bf2f_lo(kl[1][i]), dm_bf2f_hi(kh[1][i]) + dm_bf2f_hi(kl[1][i])};
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
    if (c + 1 < p.c1) load(c + 1);
    __syncthreads();
#pragma unroll
    for (int i = 0; i < 16; ++i) acc[i] *= dec;
#pragma unroll
    for (int kk = 0; kk < 4; ++kk) {
      const r_bf16x8 ah = *reinterpret_cast<const r_bf16x8*>(&Khi[wd + l32][16 * kk + 8 * lh]);
      const r_bf16x8 al = *reinterpret_cast<const r_bf16x8*>(&Klo[wd + l32][16 * kk + 8 * lh]);
      const r_bf16x8 bv = *reinterpret_cast<const r_bf16x8*>(&Vt[wj + l32][16 * kk + 8 * lh]);
      acc = __builtin_amdgcn_mfma_f32_32x32x16_bf16(ah, bv, acc, 0, 0, 0);
      acc = __builtin_amdgcn_mfma_f32_32x32x16_bf16(al, bv, acc, 0, 0, 0);
    }
    __syncthreads();
  }
#pragma unroll
  for (int q = 0; q < 4; ++q) {
    const int d = d0 + wd + 8 * q + 4 * lh;
    if (d < ds && j < p.vdim)
      *reinterpret_cast<float4*>(out + (size_t)j * ds + d) = make_float4(acc[4 * q], acc[4 * q + 1], acc[4 * q + 2], acc[4 * q + 3]);
  }
}

struct OutArgs {
  TurnedRows x;
  const bf16_t* v;
  const float* decay;
  int T, H, dim, vdim, VP, c0, c1;
  const bf16_t *s_hi, *s_lo;
  float* o;
};

// One workgroup: one chunk of one head, 32 * NV value channels. Wavefront (wq, wv) makes the outputs of
// 32 queries (two groups of sixteen) for half the channels. All products run transposed, so that a lane
// owns a query from the scores to the output: O^T = S_0 Q^T, then + V^T P^T. A product of two numbers in
// two parts each leaves out the product of their low parts.
template <int KD, int NV>
__global__ __launch_bounds__(256) void retention_out_kernel(OutArgs p) {
  constexpr int DP = KD * 32, VB = 32 * NV;
  __shared__ __attribute__((aligned(16))) bf16_t Vt[VB][LS];
  __shared__ float pw[2 * C + 1];  // powers of the decay from -64 on, zero below 0
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, l16 = lane & 15, lg = lane >> 4;
  const int c = p.c0 + blockIdx.x, h = blockIdx.z, jb = blockIdx.y * VB;
  const int wq = (wave & 1) * 32, wv = (wave >> 1) * (VB / 2);
  const int t0 = c * C;
  if (tid <= 2 * C) pw[tid] = tid < C ? 0.f : p.decay[(size_t)h * ORNITH_DECAY_POWERS + tid - C];
  // values, turned: a thread brings two tokens of eight channels
  for (int i = tid; i < (VB / 8) * (C / 2); i += 256) {
    const int oct = (i & 3) + 4 * (i >> 7), pair = (i >> 2) & 31;  // as in the scan
    const r_u32x4 zero = {0, 0, 0, 0};
    r_u32x4 a = zero, b = zero;
    if (jb + 8 * oct < p.vdim) {
      const bf16_t* src = p.v + (size_t)h * p.vdim + jb + 8 * oct;
      a = *reinterpret_cast<const r_u32x4*>(src + (size_t)min(t0 + 2 * pair, p.T - 1) * p.H * p.vdim);
      b = *reinterpret_cast<const r_u32x4*>(src + (size_t)min(t0 + 2 * pair + 1, p.T - 1) * p.H * p.vdim);
    }
    const int at = (2 * pair & 32) + vt_pos(2 * pair & 31);
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      *reinterpret_cast<uint32_t*>(&Vt[8 * oct + 2 * e][at]) = (a[e] & 0xffffu) | (b[e] << 16);
      *reinterpret_cast<uint32_t*>(&Vt[8 * oct + 2 * e + 1][at]) = (a[e] >> 16) | (b[e] & 0xffff0000u);
    }
  }
  // queries: fragment kk holds channels 32 kk + 8 lg .. of query l16
  r_bf16x8 qh[2][KD], ql[2][KD];
  int tq[2];
#pragma unroll
  for (int s = 0; s < 2; ++s) {
    tq[s] = t0 + wq + 16 * s + l16;
    const size_t row = ((size_t)min(tq[s], p.T - 1) * p.H + h) * p.dim;
#pragma unroll
    for (int kk = 0; kk < KD; ++kk) {
      const int d = 32 * kk + 8 * lg;
      r_u32x4 x = {0, 0, 0, 0}, y = x;
      if (d < p.dim) {
        x = *reinterpret_cast<const r_u32x4*>(p.x.q_hi + row + d);
        y = *reinterpret_cast<const r_u32x4*>(p.x.q_lo + row + d);
      }
      qh[s][kk] = __builtin_bit_cast(r_bf16x8, x);
      ql[s][kk] = __builtin_bit_cast(r_bf16x8, y);
    }
  }
  // the part of S_0
  const size_t cb = (size_t)h * (p.c1 - p.c0) + blockIdx.x;
  const bf16_t* sh = p.s_hi + cb * p.VP * DP;
  const bf16_t* sl = p.s_lo + cb * p.VP * DP;
  r_f32x4 acc[2][NV];
#pragma unroll
  for (int s = 0; s < 2; ++s)
#pragma unroll
    for (int vt = 0; vt < NV; ++vt) acc[s][vt] = r_f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int vt = 0; vt < NV; ++vt) {
    const size_t row = (size_t)((jb + wv) / 16 + vt) * KD * 512 + (size_t)lane * 8;
#pragma unroll
    for (int kk = 0; kk < KD; ++kk) {
      const r_bf16x8 ah = *reinterpret_cast<const r_bf16x8*>(sh + row + kk * 512);
      const r_bf16x8 al = *reinterpret_cast<const r_bf16x8*>(sl + row + kk * 512);
#pragma unroll
      for (int s = 0; s < 2; ++s) {
        acc[s][vt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(ah, qh[s][kk], acc[s][vt], 0, 0, 0);
        acc[s][vt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(al, qh[s][kk], acc[s][vt], 0, 0, 0);
        acc[s][vt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(ah, ql[s][kk], acc[s][vt], 0, 0, 0);
      }
    }
  }
  __syncthreads();
#pragma unroll
  for (int s = 0; s < 2; ++s) {
    const float x = pw[C + 1 + wq + 16 * s + l16];
#pragma unroll
    for (int vt = 0; vt < NV; ++vt) acc[s][vt] *= x;
  }
  // the chunk's own tokens, 32 at a time (none after this wavefront's last query)
#pragma unroll
  for (int half = 0; half < 2; ++half) {
    if (32 * half > wq + 31) break;
    r_f32x4 sc[2][2];
#pragma unroll
    for (int kt = 0; kt < 2; ++kt) {
#pragma unroll
      for (int s = 0; s < 2; ++s) sc[s][kt] = r_f32x4{0.f, 0.f, 0.f, 0.f};
      const size_t row = ((size_t)min(t0 + 32 * half + 16 * kt + l16, p.T - 1) * p.H + h) * p.dim;
#pragma unroll
      for (int kk = 0; kk < KD; ++kk) {
        const int d = 32 * kk + 8 * lg;
        r_u32x4 x = {0, 0, 0, 0}, y = x;
        if (d < p.dim) {
          x = *reinterpret_cast<const r_u32x4*>(p.x.k_hi + row + d);
          y = *reinterpret_cast<const r_u32x4*>(p.x.k_lo + row + d);
        }
        const r_bf16x8 kh = __builtin_bit_cast(r_bf16x8, x), kl = __builtin_bit_cast(r_bf16x8, y);
#pragma unroll
        for (int s = 0; s < 2; ++s) {
          sc[s][kt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kh, qh[s][kk], sc[s][kt], 0, 0, 0);
          sc[s][kt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kl, qh[s][kk], sc[s][kt], 0, 0, 0);
          sc[s][kt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kh, ql[s][kk], sc[s][kt], 0, 0, 0);
        }
      }
    }
    // P: key 32 half + 16 kt + 4 lg + r of query tq
    r_bf16x8 ph[2], pl[2];
#pragma unroll
    for (int s = 0; s < 2; ++s) {
      uint32_t hi[4], lo[4];
#pragma unroll
      for (int kt = 0; kt < 2; ++kt) {
        const int at = C + wq + 16 * s + l16 - (32 * half + 16 * kt + 4 * lg);
        float w[4];
#pragma unroll
        for (int r = 0; r < 4; ++r) w[r] = pw[at - r] * sc[s][kt][r];
        split2(w[0], w[1], hi[2 * kt], lo[2 * kt]);
        split2(w[2], w[3], hi[2 * kt + 1], lo[2 * kt + 1]);
      }
      const r_u32x4 hv = {hi[0], hi[1], hi[2], hi[3]}, lv = {lo[0], lo[1], lo[2], lo[3]};
      ph[s] = __builtin_bit_cast(r_bf16x8, hv);
      pl[s] = __builtin_bit_cast(r_bf16x8, lv);
    }
#pragma unroll
    for (int vt = 0; vt < NV; ++vt) {
      const r_bf16x8 vf = *reinterpret_cast<const r_bf16x8*>(&Vt[wv + 16 * vt + l16][32 * half + 8 * lg]);
#pragma unroll
      for (int s = 0; s < 2; ++s) {
        acc[s][vt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf, ph[s], acc[s][vt], 0, 0, 0);
        acc[s][vt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf, pl[s], acc[s][vt], 0, 0, 0);
      }
    }
  }
#pragma unroll
  for (int s = 0; s < 2; ++s) {
    if (tq[s] >= p.T) continue;
    float* dst = p.o + ((size_t)tq[s] * p.H + h) * p.vdim;
#pragma unroll
    for (int vt = 0; vt < NV; ++vt) {
      const int jj = jb + wv + 16 * vt + 4 * lg;
      if (jj < p.vdim)
        *reinterpret_cast<float4*>(dst + jj) = make_float4(acc[s][vt][0], acc[s][vt][1], acc[s][vt][2], acc[s][vt][3]);
    }
  }
}

template <int KD>
void launch_out(ornith_ctx* ctx, const OutArgs& p) {
  if (p.vdim <= 64)
    hipLaunchKernelGGL((retention_out_kernel<KD, 2>), dim3(p.c1 - p.c0, 1, p.H), dim3(256), 0, ctx->stream, p);
  else
    hipLaunchKernelGGL((retention_out_kernel<KD, 4>), dim3(p.c1 - p.c0, p.VP / 128, p.H), dim3(256), 0, ctx->stream, p);
}

int run_chunked(ornith_ctx* ctx, const ornith_retention_call* c, const RotArgs& rot, float kscale, float* st_out) {
  const int KD = c->dim <= 64 ? 2 : c->dim <= 128 ? 4 : 8, DP = KD * 32;
  const int VP = c->vdim <= 64 ? 64 : (c->vdim + 127) / 128 * 128;
  const int chunks = (c->T + C - 1) / C;
  // chunks a scan / output launch pair takes: what the scan writes (and the outputs read) should
  // still be in the last-level cache
  const size_t per_chunk = (size_t)c->H * VP * DP * 4;
  int block = (int)((size_t(96) << 20) / per_chunk);
  block = block < 8 ? 8 : block;
  block = block > chunks ? chunks : block;
  const size_t keys = (size_t)c->T * c->H * c->dim;
  void* base = nullptr;
  int rc = ornith_scratch(ctx, 4 * keys * 2 + per_chunk * block + 8 * 256, &base);
  if (rc) return rc;
  ScratchCursor sc(base);
  TurnedRows x;
  x.q_hi = sc.take<bf16_t>(keys);
  x.q_lo = sc.take<bf16_t>(keys);
  x.k_hi = sc.take<bf16_t>(keys);
  x.k_lo = sc.take<bf16_t>(keys);
  bf16_t* s_hi = sc.take<bf16_t>((size_t)c->H * block * VP * DP);
  bf16_t* s_lo = sc.take<bf16_t>((size_t)c->H * block * VP * DP);
  hipLaunchKernelGGL(retention_turn_kernel, dim3(c->T), dim3(NT), 0, ctx->stream, (const bf16_t*)c->d_q, (const bf16_t*)c->d_k, rot,
                     kscale, c->H, c->dim, x);
  ORN_LAUNCH_CHECK("retention_turn_kernel");
  for (int c0 = 0; c0 < chunks; c0 += block) {
    const int c1 = c0 + block < chunks ? c0 + block : chunks;
    ScanArgs s{x.k_hi, x.k_lo, (const bf16_t*)c->d_v, c->d_decay, c->T, c->H, c->dim, c->vdim, DP, VP, c0, c1,
               c0 ? st_out : c->d_state_in, st_out, s_hi, s_lo};
    hipLaunchKernelGGL(retention_scan_kernel, dim3(DP / TILE, VP / TILE, c->H), dim3(256), 0, ctx->stream, s);
    ORN_LAUNCH_CHECK("retention_scan_kernel");
    OutArgs o{x, (const bf16_t*)c->d_v, c->d_decay, c->T, c->H, c->dim, c->vdim, VP, c0, c1, s_hi, s_lo, c->d_o};
    if (KD == 2) launch_out<2>(ctx, o);
    else if (KD == 4) launch_out<4>(ctx, o);
    else launch_out<8>(ctx, o);
    ORN_LAUNCH_CHECK("retention_out_kernel");
  }
  return ORNITH_OK;
}

}  // namespace

extern "C" {

size_t ornith_retention_state_floats(int H, int dim, int vdim) { return (size_t)H * head_floats(dim, vdim); }

int ornith_decay_powers(ornith_ctx* ctx, int H, const double* decay, float* d_out) {
  ORN_REQUIRE(ctx && decay && d_out && H >= 1, "decay_powers: bad argument");
  std::vector<float> t((size_t)H * ORNITH_DECAY_POWERS);
  for (int h = 0; h < H; ++h)
    for (int n = 0; n < ORNITH_DECAY_POWERS; ++n) t[(size_t)h * ORNITH_DECAY_POWERS + n] = (float)std::pow(decay[h], n);
  return ornith_upload(ctx, d_out, t.data(), t.size() * 4);
}

int ornith_retention(ornith_ctx* ctx, const ornith_retention_call* c) {
  ORN_REQUIRE(ctx && c && c->d_q && c->d_k && c->d_v && c->d_decay && c->d_state_in && c->d_slots && c->d_o,
              "retention: null argument");
  ORN_REQUIRE(c->T >= 1 && c->H >= 1 && c->H <= 65535 && c->dim >= 1 && c->dim <= 512 && c->vdim >= 1,
              "retention: T=%d H=%d dim=%d (at most 512) vdim=%d", c->T, c->H, c->dim, c->vdim);
  ORN_REQUIRE(c->rope_dims >= 0 && c->rope_dims % 2 == 0 && c->rope_dims <= c->dim && (c->rope_dims == 0 || (c->d_cos && c->d_sin)),
              "retention: %d rotated dimensions of %d", c->rope_dims, c->dim);
  ORN_REQUIRE(c->offset >= 0 && (c->rope_dims == 0 || c->offset + c->T <= c->table_npos),
              "retention: positions [%d, %d) of a table of %d", c->offset, c->offset + c->T, c->table_npos);
  ORN_REQUIRE(c->n_slots >= 1 && c->first_slot >= 0 && c->first_slot < c->n_slots && (!c->snapshots || c->T < c->n_slots),
              "retention: slot %d of %d for %d rows", c->first_slot, c->n_slots, c->T);
  const size_t slot = ornith_retention_state_floats(c->H, c->dim, c->vdim);
  float* first = c->d_slots + (size_t)c->first_slot * slot;
  ORN_REQUIRE(first != c->d_state_in, "retention: the slot a call starts from is not one it may write");
  const RotArgs rot{c->d_cos, c->d_sin, c->rope_dims / 2, c->offset};
  const float kscale = 1.0f / __builtin_sqrtf((float)c->dim);
  if (c->act == ORNITH_BF16 && c->T >= C && !c->snapshots && ornith_option_retention_chunked() && c->dim % 8 == 0 &&
      c->vdim % 8 == 0 && c->dim <= 256)
    return run_chunked(ctx, c, rot, kscale, first);
  StepArgs p{c->d_q, c->d_k, c->d_v, rot, c->d_decay, kscale, c->T, c->H, c->dim, c->vdim, c->d_state_in, c->d_slots, slot,
             c->n_slots, c->first_slot, c->snapshots, c->d_o};
  return c->act == ORNITH_F32 ? launch_step<float>(ctx, p) : launch_step<bf16_t>(ctx, p);
}

}  // extern "C"
