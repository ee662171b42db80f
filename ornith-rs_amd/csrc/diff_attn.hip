// Differential attention (Ye et al., "Differential Transformer") over a KV cache: two softmax maps a
// head over the same values, a1 - lambda a2, a norm over the head and a gate, with rotary positions, a
// sliding window and kept first tokens. The arithmetic is stated at ornith_diff_attn in ornith_hip.h.
//
// Decode widths (and 32-bit models): a query's visible keys, kept first tokens and window one after the
// other, are cut into blocks; a workgroup takes one block of one KV head for all its query heads and
// both maps. It turns the query and the call's new keys itself (what it stages instead of the cache's
// not yet written rows, and stores to the cache as a side effect), so a layer's attention is one launch
// while a query has a single block, and a merge launch more otherwise.
//
// Prefill widths (bf16): a launch that rotates queries and appends keys and values, then flash attention
// on the matrix cores with both maps in one pass: a value fragment read from LDS serves both.
#include "act_device.h"
#include "mfma_device.h"
#include "rt.h"

namespace {

struct DaArgs {
  const void *q, *k, *v;
  const float* gate;
  const float *cos_t, *sin_t;
  int rope_half;
  int T, H, G, dim, vdim, offset, cap, window, keep;
  float scale, lambda, diff, eps;
  void *k_cache, *v_cache, *q_rot, *out;
};

// what the query at position pos sees: keys [0, head) and [lo, pos]
__device__ __forceinline__ void visible(const DaArgs& p, int pos, int& head, int& lo) {
  lo = p.window > 0 ? max(0, pos - p.window + 1) : 0;
  head = min(p.keep, lo);
}

// element d of one map's row at position pos, rotated: what it is made of (loads only), then itself
template <typename A>
struct Turn {
  A x, y;
  float c, s;
  bool on;
  __device__ __forceinline__ void load(const A* row, int d, int pos, const DaArgs& p) {
    on = d < 2 * p.rope_half;
    x = row[d];
    y = x;
    c = 1.f;
    s = 0.f;
    if (on) {
      y = row[d ^ 1];
      const size_t at = (size_t)pos * p.rope_half + (d >> 1);
      c = p.cos_t[at];
      s = p.sin_t[at];
    }
  }
  __device__ __forceinline__ A value(int d) const {
    if (!on) return x;
    const float a = act_f(x), b = act_f(y);
    return act_of<A>((d & 1) ? dm_fma(b, s, a * c) : dm_fma(-b, s, a * c));
  }
};

constexpr int NT = 256;

// The end of a head, by one wavefront: a1 - lambda a2 (columns lane, lane + 64, ..), its norm, the gate.
template <typename A, typename F>
__device__ __forceinline__ void finish_head(const DaArgs& p, int t, int h, int lane, F diff_at) {
  float ss = 0.f;
  for (int c = lane; c < p.vdim; c += 64) {
    const float o = diff_at(c);
    ss = dm_fma(o, o, ss);
  }
  const float inv = dm_rsqrt(dm_wave_sum<64>(ss) / (float)p.vdim + p.eps);
  const float g = (1.0f - p.diff) * dm_sigmoid_f32(p.gate[(size_t)t * p.H + h]);
  A* dst = reinterpret_cast<A*>(p.out) + ((size_t)t * p.H + h) * p.vdim;
  for (int c = lane; c < p.vdim; c += 64) dst[c] = act_of<A>((diff_at(c) * inv) * g);
}

// ---- decode widths ---------------------------------------------------------------------
// grid (blocks, G, rows); KB keys a block. part: f32 [rows][H][2][blocks][vdim], ml: [rows][H][2][blocks][2]
template <typename A, bool VEC>
__global__ __launch_bounds__(NT) void diff_decode_kernel(DaArgs p, int KB, int t_base, float* part, float* ml) {
  extern __shared__ __attribute__((aligned(16))) char lds_raw[];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int R = p.H / p.G, rows = 2 * R, kd = 2 * p.dim;
  const int g = blockIdx.y, t = t_base + blockIdx.z, pos = p.offset + t, blocks = gridDim.x;
  int head, lo;
  visible(p, pos, head, lo);
  const int nvis = head + pos - lo + 1, u0 = blockIdx.x * KB;
  if (u0 >= nvis) return;  // (every thread of the workgroup)
  const int nk = min(KB, nvis - u0);
  const int qd = (p.dim + 3) & ~3, kst = ((kd + 7) & ~7) + 16 / (int)sizeof(A), vst = (p.vdim + 7) & ~7;
  float* qs = reinterpret_cast<float*>(lds_raw);  // [rows][qd]
  float* sc = qs + rows * qd;                     // [rows][KB]
  float* os = sc + rows * KB;                     // [rows][vdim rounded up to 4]
  const int ost = (p.vdim + 3) & ~3;
  A* ks = reinterpret_cast<A*>(os + rows * ost);  // [KB][kst]
  A* vs = ks + (size_t)KB * kst;                  // [KB][vst]

  // what is staged: the group's queries, rotated (row 2 r + map of head g R + r), the block's cached keys
  // and values, and the call's own
  const A* kc = reinterpret_cast<const A*>(p.k_cache) + (size_t)g * p.cap * kd;
  const A* vc = reinterpret_cast<const A*>(p.v_cache) + (size_t)g * p.cap * p.vdim;
  auto key_at = [&](int i) { const int u = u0 + i; return u < head ? u : lo + (u - head); };
  // the call's own keys among the block's: always its last ones
  int r_new = nk;
  for (int r = max(0, nk - (pos - p.offset + 1)); r < nk; ++r)
    if (key_at(r) >= p.offset) {
      r_new = r;
      break;
    }
  const int n_new = (nk - r_new) * kd, n_q = rows * qd;
  auto q_row = [&](int r) { return reinterpret_cast<const A*>(p.q) + (((size_t)t * p.H + g * R + (r >> 1)) * 2 + (r & 1)) * p.dim; };
  auto new_row = [&](int j, int m) { return reinterpret_cast<const A*>(p.k) + (((size_t)(j - p.offset) * p.G + g) * 2 + m) * p.dim; };
  // (queries as the prefill path keeps them: rotated, an activation again)
  auto put_q = [&](int i, const Turn<A>& u) { const int d = i % qd; qs[i] = d < p.dim ? act_f(u.value(d)) : 0.f; };
  auto load_q = [&](int i, Turn<A>& u) { const int d = i % qd; if (d < p.dim) u.load(q_row(i / qd), d, pos, p); };
  auto load_new = [&](int i, Turn<A>& u) {
    const int c = i % kd, m = c >= p.dim ? 1 : 0, j = key_at(r_new + i / kd);
    u.load(new_row(j, m), c - m * p.dim, j, p);
  };
  auto put_new = [&](int i, const Turn<A>& u) {
    const int r = r_new + i / kd, c = i % kd, j = key_at(r);
    const A x = u.value(c >= p.dim ? c - p.dim : c);
    ks[r * kst + c] = x;
    if (j == pos) reinterpret_cast<A*>(p.k_cache)[((size_t)g * p.cap + j) * kd + c] = x;
  };
  auto v_row = [&](int j) {
    return j < p.offset ? vc + (size_t)j * p.vdim : reinterpret_cast<const A*>(p.v) + ((size_t)(j - p.offset) * p.G + g) * p.vdim;
  };
  // everything a thread stages first is asked for before any of it is waited for
  constexpr int QB = 2;
  Turn<A> qu[QB], nu;
#pragma unroll
  for (int b = 0; b < QB; ++b)
    if (tid + NT * b < n_q) load_q(tid + NT * b, qu[b]);
  if (tid < n_new) load_new(tid, nu);
  if constexpr (VEC) {
    constexpr int E = 16 / (int)sizeof(A), B = 4;
    const int kch = kd / E, vch = p.vdim / E, nkc = r_new * kch, nvc = nk * vch;
    uint4 kr[B], vr[B];
    auto k_piece = [&](int i) { return *reinterpret_cast<const uint4*>(kc + (size_t)key_at(i / kch) * kd + (i % kch) * E); };
    auto v_piece = [&](int i) { return *reinterpret_cast<const uint4*>(v_row(key_at(i / vch)) + (i % vch) * E); };
#pragma unroll
    for (int b = 0; b < B; ++b)
      if (tid + NT * b < nkc) kr[b] = k_piece(tid + NT * b);
#pragma unroll
    for (int b = 0; b < B; ++b)
      if (tid + NT * b < nvc) vr[b] = v_piece(tid + NT * b);
#pragma unroll
    for (int b = 0; b < B; ++b) {
      const int i = tid + NT * b;
      if (i < nkc) *reinterpret_cast<uint4*>(&ks[(i / kch) * kst + (i % kch) * E]) = kr[b];
    }
#pragma unroll
    for (int b = 0; b < B; ++b) {
      const int i = tid + NT * b;
      if (i < nvc) *reinterpret_cast<uint4*>(&vs[(i / vch) * vst + (i % vch) * E]) = vr[b];
    }
    for (int i = tid + NT * B; i < nkc; i += NT) *reinterpret_cast<uint4*>(&ks[(i / kch) * kst + (i % kch) * E]) = k_piece(i);
    for (int i = tid + NT * B; i < nvc; i += NT) *reinterpret_cast<uint4*>(&vs[(i / vch) * vst + (i % vch) * E]) = v_piece(i);
  } else {
    for (int i = tid; i < r_new * kd; i += NT) ks[(i / kd) * kst + i % kd] = kc[(size_t)key_at(i / kd) * kd + i % kd];
    for (int i = tid; i < nk * p.vdim; i += NT) vs[(i / p.vdim) * vst + i % p.vdim] = v_row(key_at(i / p.vdim))[i % p.vdim];
  }
#pragma unroll
  for (int b = 0; b < QB; ++b)
    if (tid + NT * b < n_q) put_q(tid + NT * b, qu[b]);
  for (int i = tid + NT * QB; i < n_q; i += NT) {
    Turn<A> u{};
    load_q(i, u);
    put_q(i, u);
  }
  if (tid < n_new) put_new(tid, nu);
  for (int i = tid + NT; i < n_new; i += NT) {
    Turn<A> u;
    load_new(i, u);
    put_new(i, u);
  }
  // this query's own value row
  if (r_new < nk && key_at(nk - 1) == pos)
    for (int c = tid; c < p.vdim; c += NT)
      reinterpret_cast<A*>(p.v_cache)[((size_t)g * p.cap + pos) * p.vdim + c] =
          reinterpret_cast<const A*>(p.v)[((size_t)t * p.G + g) * p.vdim + c];
  __syncthreads();

  // scores: a thread takes one key and every (NT / KB)-th row
  {
    const int key = tid % KB, step = NT / KB;
    for (int r = tid / KB; r < rows; r += step) {
      float s = -DM_INF;
      if (key < nk) {
        const A* kr = &ks[key * kst + (r & 1) * p.dim];
        const float* qr = qs + r * qd;
        s = 0.f;
        if constexpr (VEC) {
#pragma unroll 8
          for (int d = 0; d < p.dim; d += 4) {
            float kv[4];
            act_load<4>(kr + d, kv);
            const float4 q4 = *reinterpret_cast<const float4*>(qr + d);
            s = dm_fma(kv[3], q4.w, dm_fma(kv[2], q4.z, dm_fma(kv[1], q4.y, dm_fma(kv[0], q4.x, s))));
          }
        } else {
          for (int d = 0; d < p.dim; ++d) s = dm_fma(act_f(kr[d]), qr[d], s);
        }
        s *= p.scale;
      }
      sc[r * KB + key] = s;
    }
  }
  __syncthreads();
  // a row's maximum, exponentials and sum: one wavefront a row
  for (int r = wave; r < rows; r += NT / 64) {
    const float s = lane < KB ? sc[r * KB + lane] : -DM_INF;
    const float m = dm_wave_max<64>(s);
    const float e = s == -DM_INF ? 0.f : dm_exp(s - m);
    const float l = dm_wave_sum<64>(e);
    if (lane < KB) sc[r * KB + lane] = e;
    if (lane == 0) {
      const int h = g * R + (r >> 1);
      if (blocks > 1) {
        float* d = ml + ((((size_t)blockIdx.z * p.H + h) * 2 + (r & 1)) * blocks + blockIdx.x) * 2;
        d[0] = m;
        d[1] = l;
      }
      qs[r * qd] = 1.0f / l;  // (the queries are done with)
    }
  }
  __syncthreads();
  // weighted values: a thread takes one row and a run of columns
  {
    constexpr int W = VEC ? 4 : 1;
    const int cols = p.vdim / W;
    for (int i = tid; i < rows * cols; i += NT) {
      const int r = i / cols, c = (i % cols) * W;
      float o[W];
#pragma unroll
      for (int e = 0; e < W; ++e) o[e] = 0.f;
      const float* pr = sc + r * KB;
#pragma unroll 16
      for (int key = 0; key < nk; ++key) {
        const float w = pr[key];
        if constexpr (VEC) {
          float vv[4];
          act_load<4>(&vs[key * vst + c], vv);
#pragma unroll
          for (int e = 0; e < W; ++e) o[e] = dm_fma(w, vv[e], o[e]);
        } else {
          o[0] = dm_fma(w, act_f(vs[key * vst + c]), o[0]);
        }
      }
      if (blocks > 1) {
        float* d = part + ((((size_t)blockIdx.z * p.H + g * R + (r >> 1)) * 2 + (r & 1)) * blocks + blockIdx.x) * p.vdim + c;
#pragma unroll
        for (int e = 0; e < W; ++e) d[e] = o[e];
      } else {
        const float inv = qs[r * qd];
#pragma unroll
        for (int e = 0; e < W; ++e) os[r * ost + c + e] = o[e] * inv;
      }
    }
  }
  if (blocks > 1) return;
  __syncthreads();
  for (int r = wave; r < R; r += NT / 64)
    finish_head<A>(p, t, g * R + r, lane, [&](int c) { return os[2 * r * ost + c] - p.lambda * os[(2 * r + 1) * ost + c]; });
}

// The blocks of a query joined. grid (H, rows): blocks in ascending order with weights e^(m_b - M).
template <typename A>
__global__ __launch_bounds__(NT) void diff_merge_kernel(DaArgs p, int KB, int t_base, int stride, const float* part, const float* ml) {
  extern __shared__ __attribute__((aligned(16))) char lds_raw[];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int h = blockIdx.x, t = t_base + blockIdx.y, pos = p.offset + t;
  int head, lo;
  visible(p, pos, head, lo);
  const int nb = (head + pos - lo + 1 + KB - 1) / KB;
  float* wb = reinterpret_cast<float*>(lds_raw);  // [2][stride]
  float* os = wb + 2 * stride;                    // [2][vdim]
  const size_t base = ((size_t)blockIdx.y * p.H + h) * 2 * stride;
  if (wave < 2) {
    const float* mr = ml + (base + (size_t)wave * stride) * 2;
    float M = -DM_INF;
    for (int b = lane; b < nb; b += 64) M = __builtin_fmaxf(M, mr[2 * b]);
    M = dm_wave_max<64>(M);
    float L = 0.f;
    for (int b = lane; b < nb; b += 64) {
      const float w = dm_exp(mr[2 * b] - M);
      wb[wave * stride + b] = w;
      L = dm_fma(w, mr[2 * b + 1], L);
    }
    L = dm_wave_sum<64>(L);
    for (int b = lane; b < nb; b += 64) wb[wave * stride + b] = wb[wave * stride + b] / L;
  }
  __syncthreads();
  for (int i = tid; i < 2 * p.vdim; i += NT) {
    const int m = i / p.vdim, c = i % p.vdim;
    const float* src = part + (base + (size_t)m * stride) * p.vdim + c;
    const float* w = wb + m * stride;
    float o = 0.f;
    int b = 0;
    for (; b + 16 <= nb; b += 16) {
      float x[16];
#pragma unroll
      for (int e = 0; e < 16; ++e) x[e] = src[(size_t)(b + e) * p.vdim];
#pragma unroll
      for (int e = 0; e < 16; ++e) o = dm_fma(w[b + e], x[e], o);
    }
    for (; b < nb; ++b) o = dm_fma(w[b], src[(size_t)b * p.vdim], o);
    os[i] = o;
  }
  __syncthreads();
  if (wave == 0) finish_head<A>(p, t, h, lane, [&](int c) { return os[c] - p.lambda * os[p.vdim + c]; });
}

template <typename A>
int run_decode(ornith_ctx* ctx, const DaArgs& p) {
  const int R = p.H / p.G, rows = 2 * R, kd = 2 * p.dim;
  const bool vec = p.dim % 4 == 0 && kd % (16 / (int)sizeof(A)) == 0 && p.vdim % (16 / (int)sizeof(A)) == 0;
  const size_t qd = (p.dim + 3) & ~3, ost = (p.vdim + 3) & ~3;
  const size_t key = ((size_t)((kd + 7) & ~7) + 16 / sizeof(A) + ((p.vdim + 7) & ~7)) * sizeof(A) + rows * 4;
  int KB = 64;
  auto lds_of = [&](int kb) { return (rows * (qd + ost)) * 4 + (size_t)kb * key; };
  while (KB > 16 && lds_of(KB) > 65536) KB /= 2;
  const size_t lds = lds_of(KB);
  ORN_REQUIRE(lds <= 160 * 1024, "diff_attn: %d heads of %d + %d values a KV head do not fit a compute unit's local memory", R,
              2 * p.dim, p.vdim);
  const int last = p.offset + p.T - 1;
  const int most = p.window > 0 ? (last + 1 < p.window + p.keep ? last + 1 : p.window + p.keep) : last + 1;
  const int blocks = (most + KB - 1) / KB;
  if (lds > 65536) {
    ORN_HIP(hipFuncSetAttribute((const void*)diff_decode_kernel<A, true>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds));
    ORN_HIP(hipFuncSetAttribute((const void*)diff_decode_kernel<A, false>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds));
  }
  // rows in groups whose partial results stay below 256 MB
  int group = p.T < 32768 ? p.T : 32768;
  float *part = nullptr, *ml = nullptr;
  if (blocks > 1) {
    const size_t per = (size_t)p.H * 2 * blocks * (p.vdim + 2) * 4;
    const size_t fit = (size_t(256) << 20) / per;
    if ((size_t)group > fit) group = fit < 1 ? 1 : (int)fit;
    void* base = nullptr;
    const int rc = ornith_scratch(ctx, per * group + 1024, &base);
    if (rc) return rc;
    ScratchCursor sc(base);
    part = sc.take<float>((size_t)group * p.H * 2 * blocks * p.vdim);
    ml = sc.take<float>((size_t)group * p.H * 2 * blocks * 2);
  }
  for (int t = 0; t < p.T; t += group) {
    const int n = p.T - t < group ? p.T - t : group;
    if (vec)
      hipLaunchKernelGGL((diff_decode_kernel<A, true>), dim3(blocks, p.G, n), dim3(NT), lds, ctx->stream, p, KB, t, part, ml);
    else
      hipLaunchKernelGGL((diff_decode_kernel<A, false>), dim3(blocks, p.G, n), dim3(NT), lds, ctx->stream, p, KB, t, part, ml);
    ORN_LAUNCH_CHECK("diff_decode_kernel");
    if (blocks > 1) {
      hipLaunchKernelGGL(diff_merge_kernel<A>, dim3(p.H, n), dim3(NT), (2 * (size_t)blocks + 2 * (size_t)p.vdim) * 4, ctx->stream, p,
                         KB, t, blocks, part, ml);
      ORN_LAUNCH_CHECK("diff_merge_kernel");
    }
  }
  return ORNITH_OK;
}

// ---- prefill widths ----------------------------------------------------------------------
// queries rotated into q_rot, keys rotated and values as they are into the cache; a thread takes eight
// elements (four pairs), grid.x the rows
__global__ __launch_bounds__(NT) void diff_prep_kernel(DaArgs p) {
  const int t = blockIdx.x, pos = p.offset + t, per = p.dim / 8, vper = p.vdim / 8;
  const int nq = p.H * 2 * per, nk = p.G * 2 * per, nv = p.G * vper;
  const float* ct = p.cos_t + (size_t)pos * p.rope_half;
  const float* st = p.sin_t + (size_t)pos * p.rope_half;
  for (int i = threadIdx.x; i < nq + nk + nv; i += NT) {
    if (i >= nq + nk) {
      const int e = i - nq - nk, g = e / vper, c = 8 * (e % vper);
      *reinterpret_cast<uint4*>(reinterpret_cast<bf16_t*>(p.v_cache) + ((size_t)g * p.cap + pos) * p.vdim + c) =
          *reinterpret_cast<const uint4*>(reinterpret_cast<const bf16_t*>(p.v) + ((size_t)t * p.G + g) * p.vdim + c);
      continue;
    }
    const bool is_q = i < nq;
    const int a = is_q ? i : i - nq, row = a / per, d = 8 * (a % per);
    const bf16_t* src = is_q ? reinterpret_cast<const bf16_t*>(p.q) + (size_t)t * p.H * 2 * p.dim
                             : reinterpret_cast<const bf16_t*>(p.k) + (size_t)t * p.G * 2 * p.dim;
    const uint4 in = *reinterpret_cast<const uint4*>(src + (size_t)row * p.dim + d);
    uint32_t w[4] = {in.x, in.y, in.z, in.w};
#pragma unroll
    for (int e = 0; e < 4; ++e)
      if (d + 2 * e < 2 * p.rope_half) {
        const float c = ct[(d >> 1) + e], s = st[(d >> 1) + e], x = dm_bf2f_lo(w[e]), y = dm_bf2f_hi(w[e]);
        w[e] = dm_f2bf2(dm_fma(-y, s, x * c), dm_fma(x, s, y * c));
      }
    bf16_t* dst = is_q ? reinterpret_cast<bf16_t*>(p.q_rot) + ((size_t)t * p.H * 2 + row) * p.dim + d
                       : reinterpret_cast<bf16_t*>(p.k_cache) + ((size_t)(row >> 1) * p.cap + pos) * 2 * p.dim + (row & 1) * p.dim + d;
    *reinterpret_cast<uint4*>(dst) = make_uint4(w[0], w[1], w[2], w[3]);
  }
}

typedef __bf16 d_bf16x8 __attribute__((ext_vector_type(8)));
typedef float d_f32x4 __attribute__((ext_vector_type(4)));
typedef uint32_t d_u32x4 __attribute__((ext_vector_type(4)));

constexpr int BQ = 64, BKV = 64, LV = BKV + 8;

// One workgroup: 64 query rows of one head, sixteen a wavefront. Both products run transposed
// (S^T = K Q^T, O^T += V^T P^T): a lane owns a query from the scores to the output and the weights never
// leave the registers. They go to the matrix cores as two bf16 parts, so they count as 32-bit numbers.
// KD: 32-channel steps of a map; VT: 16-channel tiles of the values.
template <int KD, int VT>
__global__ __launch_bounds__(256, VT <= 8 && KD <= 2 ? 2 : 1) void diff_prefill_kernel(DaArgs p) {
  constexpr int DP = KD * 32, LK = 2 * DP + 8;
  __shared__ __attribute__((aligned(16))) bf16_t Ks[BKV][LK];
  __shared__ __attribute__((aligned(16))) bf16_t Vt[VT * 16][LV];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, l16 = lane & 15, lg = lane >> 4;
  // the last rows of a call see the most: they start first
  const int qt = gridDim.y - 1 - blockIdx.y, h = blockIdx.x, g = h / (p.H / p.G);
  const int t0 = qt * BQ, tq = t0 + wave * 16 + l16, tc = min(tq, p.T - 1), pos = p.offset + tc;
  const int first = p.offset + t0, last = p.offset + min(t0 + BQ, p.T) - 1;
  const int kd = 2 * p.dim;
  d_bf16x8 qf[2][KD];
#pragma unroll
  for (int m = 0; m < 2; ++m)
#pragma unroll
    for (int kk = 0; kk < KD; ++kk) {
      const int d = 32 * kk + 8 * lg;
      d_u32x4 x = {0, 0, 0, 0};
      if (d < p.dim)
        x = *reinterpret_cast<const d_u32x4*>(reinterpret_cast<const bf16_t*>(p.q_rot) + (((size_t)tc * p.H + h) * 2 + m) * p.dim + d);
      if (p.scale < 0.f) x ^= 0x80008000u;  // the scale's sign, so that a row's largest score is its largest product
      qf[m][kk] = __builtin_bit_cast(d_bf16x8, x);
    }
  d_f32x4 acc[2][VT];
  float mx[2], sum[2];
#pragma unroll
  for (int m = 0; m < 2; ++m) {
    mx[m] = -DM_INF;
    sum[m] = 0.f;
#pragma unroll
    for (int v = 0; v < VT; ++v) acc[m][v] = d_f32x4{0.f, 0.f, 0.f, 0.f};
  }
  const bf16_t* kc = reinterpret_cast<const bf16_t*>(p.k_cache) + (size_t)g * p.cap * kd;
  const bf16_t* vc = reinterpret_cast<const bf16_t*>(p.v_cache) + (size_t)g * p.cap * p.vdim;
  const float s2 = __builtin_fmaxf(__builtin_fabsf(p.scale) * 1.44269504088896341f, 1e-30f);
  // key blocks: the kept first tokens that lie before the window of the first row, then the window
  const int lo = p.window > 0 ? max(0, first - p.window + 1) : 0, wb0 = lo / BKV, wb1 = last / BKV;
  const int hb = min((p.keep + BKV - 1) / BKV, wb0);
  const int nblocks = hb + wb1 - wb0 + 1;
  // this thread's pieces of a key block: 16 bytes of a key row each, and pairs of value rows, turned on
  // their way into LDS; the next block's are asked for before this one is worked on. Value piece e: four
  // neighbouring lanes read 64 bytes of a row, and the sixteen row pairs of a wavefront keep its LDS
  // writes two to a bank. Offsets inside a block are made once: a block costs the vector ALU nothing here.
  constexpr int KI = 2 * KD, VI = VT / 4;
  d_u32x4 kreg[KI], vreg[VI][2];
  int krow[KI], kcol[KI], vrow[VI], vcol[VI], koff[KI], voff[VI][2];
  bool kin[KI], vin[VI];
#pragma unroll
  for (int i = 0; i < KI; ++i) {
    const int e = tid + 256 * i, c = e % (8 * KD), m = c / (4 * KD), d = 8 * (c % (4 * KD));
    krow[i] = e / (8 * KD);
    kin[i] = d < p.dim;
    kcol[i] = kin[i] ? m * p.dim + d : 0;
    koff[i] = krow[i] * kd + kcol[i];
  }
#pragma unroll
  for (int i = 0; i < VI; ++i) {
    const int e = tid + 256 * i, d = 8 * ((e & 3) + 4 * (e >> 7));
    vrow[i] = 2 * ((e >> 2) & 31);
    vin[i] = d < p.vdim;
    vcol[i] = vin[i] ? d : 0;
#pragma unroll
    for (int b = 0; b < 2; ++b) voff[i][b] = (vrow[i] + b) * p.vdim + vcol[i];
  }
  auto fetch = [&](int j0) {
    const bf16_t* kb = kc + (size_t)j0 * kd;
    const bf16_t* vb = vc + (size_t)j0 * p.vdim;
    if (j0 + BKV - 1 <= last) {
#pragma unroll
      for (int i = 0; i < KI; ++i) kreg[i] = *reinterpret_cast<const d_u32x4*>(kb + koff[i]);
#pragma unroll
      for (int i = 0; i < VI; ++i)
#pragma unroll
        for (int b = 0; b < 2; ++b) vreg[i][b] = *reinterpret_cast<const d_u32x4*>(vb + voff[i][b]);
    } else {  // the block the call's last keys end in: nothing is read past them
      const int n = last - j0;
#pragma unroll
      for (int i = 0; i < KI; ++i) kreg[i] = *reinterpret_cast<const d_u32x4*>(kb + min(krow[i], n) * kd + kcol[i]);
#pragma unroll
      for (int i = 0; i < VI; ++i)
#pragma unroll
        for (int b = 0; b < 2; ++b) vreg[i][b] = *reinterpret_cast<const d_u32x4*>(vb + min(vrow[i] + b, n) * p.vdim + vcol[i]);
    }
  };
  auto block_at = [&](int ib) { return (ib < hb ? ib : wb0 + ib - hb) * BKV; };
  const unsigned win = p.window > 0 ? (unsigned)p.window : 0x7fffffffu;
  // padding channels of the tiles stay zero
  if (p.dim < DP)
    for (int i = tid; i < BKV * LK / 8; i += 256) reinterpret_cast<uint4*>(&Ks[0][0])[i] = make_uint4(0, 0, 0, 0);
  if (p.vdim < VT * 16)
    for (int i = tid; i < VT * 16 * LV / 8; i += 256) reinterpret_cast<uint4*>(&Vt[0][0])[i] = make_uint4(0, 0, 0, 0);
  fetch(block_at(0));
  for (int ib = 0; ib < nblocks; ++ib) {
    const int j0 = block_at(ib);
    __syncthreads();
#pragma unroll
    for (int i = 0; i < KI; ++i)
      if (kin[i]) *reinterpret_cast<d_u32x4*>(&Ks[krow[i]][8 * ((tid + 256 * i) % (8 * KD))]) = kreg[i];
#pragma unroll
    for (int i = 0; i < VI; ++i)
      if (vin[i]) {
        const int at = (vrow[i] & 32) + vt_pos(vrow[i] & 31);
#pragma unroll
        for (int w = 0; w < 4; ++w) {
          *reinterpret_cast<uint32_t*>(&Vt[vcol[i] + 2 * w][at]) = __builtin_amdgcn_perm(vreg[i][1][w], vreg[i][0][w], 0x05040100u);
          *reinterpret_cast<uint32_t*>(&Vt[vcol[i] + 2 * w + 1][at]) = __builtin_amdgcn_perm(vreg[i][1][w], vreg[i][0][w], 0x07060302u);
        }
      }
    __syncthreads();
    if (ib + 1 < nblocks) fetch(block_at(ib + 1));
    // scores: key j0 + 16 kt + 4 lg + r of this lane's query. All fragments of a map are asked for before
    // the first is used, the second map's before the first map's products (left to itself the compiler
    // puts every read right before its use, an LDS latency a product)
    d_f32x4 sc[2][4];
    constexpr int GK = KD <= 2 ? 4 : VT <= 8 ? 2 : 1;  // key tiles asked for together
    d_bf16x8 kf[2][GK][KD];
    auto key_frags = [&](int step) {  // step: map, then group of key tiles
      const int m = step / (4 / GK), k0 = step % (4 / GK) * GK;
#pragma unroll
      for (int kt = 0; kt < GK; ++kt)
#pragma unroll
        for (int kk = 0; kk < KD; ++kk)
          kf[step & 1][kt][kk] = *reinterpret_cast<const d_bf16x8*>(&Ks[16 * (k0 + kt) + l16][m * DP + 32 * kk + 8 * lg]);
    };
    auto products = [&](int step) {
      const int m = step / (4 / GK), k0 = step % (4 / GK) * GK;
#pragma unroll
      for (int kt = 0; kt < GK; ++kt) sc[m][k0 + kt] = d_f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
      for (int kk = 0; kk < KD; ++kk)
#pragma unroll
        for (int kt = 0; kt < GK; ++kt)
          sc[m][k0 + kt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf[step & 1][kt][kk], qf[m][kk], sc[m][k0 + kt], 0, 0, 0);
    };
    constexpr int STEPS = 2 * (4 / GK);
    key_frags(0);
#pragma unroll
    for (int step = 0; step < STEPS; ++step) {
      __builtin_amdgcn_sched_barrier(0);
      if (step + 1 < STEPS) key_frags(step + 1);
      __builtin_amdgcn_sched_barrier(0);
      products(step);
    }
    // the first value fragments come in under the softmax
    constexpr int AHEAD = VT <= 8 ? 2 : 1;
    d_bf16x8 vf[AHEAD + 1][2];
    auto value_frags = [&](int v) {
#pragma unroll
      for (int a = 0; a < 2; ++a) vf[v % (AHEAD + 1)][a] = *reinterpret_cast<const d_bf16x8*>(&Vt[16 * v + l16][32 * a + 8 * lg]);
    };
    __builtin_amdgcn_sched_barrier(0);
#pragma unroll
    for (int v = 0; v < AHEAD; ++v) value_frags(v);
    __builtin_amdgcn_sched_barrier(0);
    // every row of the tile sees the whole block: inside everyone's window, before everyone
    const bool whole = j0 + BKV - 1 <= first && (p.window <= 0 || last - j0 < p.window || j0 + BKV <= p.keep);
    if (!whole) {
      const bool kept = j0 < p.keep;
#pragma unroll
      for (int kt = 0; kt < 4; ++kt)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int j = j0 + 16 * kt + 4 * lg + r, back = pos - j;
          bool see = (unsigned)back < win;
          if (kept) see = see | ((j < p.keep) & (back >= 0));
#pragma unroll
          for (int m = 0; m < 2; ++m) sc[m][kt][r] = see ? sc[m][kt][r] : -DM_INF;
        }
    }
    d_bf16x8 ph[2][2], pl[2][2];
#pragma unroll
    for (int m = 0; m < 2; ++m) {
      float top = sc[m][0][0];
#pragma unroll
      for (int kt = 0; kt < 4; ++kt)
#pragma unroll
        for (int r = 0; r < 4; ++r) top = __builtin_fmaxf(top, sc[m][kt][r]);
      top = dm_max_groups16(top) * s2;
      // the reference point of a row's exponentials moves only when its maximum has grown by 2^8 (the
      // weights stay below 2^8 then, the sums far inside fp32's range)
      if (__any(top > mx[m] + 8.0f)) {
        const float mn = __builtin_fmaxf(mx[m], top), alpha = mn == -DM_INF ? 0.f : dm_exp2_hw(mx[m] - mn);
        mx[m] = mn;
        sum[m] *= alpha;
#pragma unroll
        for (int v = 0; v < VT; ++v) acc[m][v] *= alpha;
      }
      const float ref = mx[m] == -DM_INF ? 0.f : mx[m];
      float l = 0.f;
#pragma unroll
      for (int a = 0; a < 2; ++a) {
        uint32_t hi[4], lo2[4];
#pragma unroll
        for (int b = 0; b < 2; ++b) {
          float e[4];
#pragma unroll
          for (int r = 0; r < 4; ++r) {
            e[r] = dm_exp2_hw(dm_fma(sc[m][2 * a + b][r], s2, -ref));
            l += e[r];
          }
          split2(e[0], e[1], hi[2 * b], lo2[2 * b]);
          split2(e[2], e[3], hi[2 * b + 1], lo2[2 * b + 1]);
        }
        const d_u32x4 hv = {hi[0], hi[1], hi[2], hi[3]}, lv = {lo2[0], lo2[1], lo2[2], lo2[3]};
        ph[m][a] = __builtin_bit_cast(d_bf16x8, hv);
        pl[m][a] = __builtin_bit_cast(d_bf16x8, lv);
      }
      sum[m] += l;
    }
#pragma unroll
    for (int v = 0; v < VT; ++v) {
      if (v + AHEAD < VT) value_frags(v + AHEAD);
      __builtin_amdgcn_sched_barrier(0);
#pragma unroll
      for (int a = 0; a < 2; ++a)
#pragma unroll
        for (int m = 0; m < 2; ++m) acc[m][v] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf[v % (AHEAD + 1)][a], ph[m][a], acc[m][v], 0, 0, 0);
#pragma unroll
      for (int a = 0; a < 2; ++a)
#pragma unroll
        for (int m = 0; m < 2; ++m) acc[m][v] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf[v % (AHEAD + 1)][a], pl[m][a], acc[m][v], 0, 0, 0);
      __builtin_amdgcn_sched_barrier(0);
    }
  }
  // a1 - lambda a2, its norm over the head (padding channels are zero), the gate
  const float i1 = 1.0f / dm_sum_groups16(sum[0]), i2 = p.lambda / dm_sum_groups16(sum[1]);
  float ss = 0.f;
#pragma unroll
  for (int v = 0; v < VT; ++v)
#pragma unroll
    for (int r = 0; r < 4; ++r) {
      const float o = acc[0][v][r] * i1 - acc[1][v][r] * i2;
      acc[0][v][r] = o;
      ss = dm_fma(o, o, ss);
    }
  const float inv = dm_rsqrt(dm_sum_groups16(ss) / (float)p.vdim + p.eps);
  if (tq >= p.T) return;
  const float gt = inv * ((1.0f - p.diff) * dm_sigmoid_f32(p.gate[(size_t)tq * p.H + h]));
  bf16_t* dst = reinterpret_cast<bf16_t*>(p.out) + ((size_t)tq * p.H + h) * p.vdim;
#pragma unroll
  for (int v = 0; v < VT; ++v) {
    const int c = 16 * v + 4 * lg;
    if (c < p.vdim) {
      const float o[4] = {acc[0][v][0] * gt, acc[0][v][1] * gt, acc[0][v][2] * gt, acc[0][v][3] * gt};
      act_store4(dst + c, o);
    }
  }
}

template <int KD>
void launch_prefill(ornith_ctx* ctx, const DaArgs& p) {
  const dim3 grid(p.H, (p.T + BQ - 1) / BQ);
  if (p.vdim <= 64)
    hipLaunchKernelGGL((diff_prefill_kernel<KD, 4>), grid, dim3(256), 0, ctx->stream, p);
  else if (p.vdim <= 128)
    hipLaunchKernelGGL((diff_prefill_kernel<KD, 8>), grid, dim3(256), 0, ctx->stream, p);
  else
    hipLaunchKernelGGL((diff_prefill_kernel<KD, 16>), grid, dim3(256), 0, ctx->stream, p);
}

}  // namespace

extern "C" int ornith_diff_attn(ornith_ctx* ctx, const ornith_diff_attn_call* c) {
  ORN_REQUIRE(ctx && c && c->d_q && c->d_k && c->d_v && c->d_gate && c->d_k_cache && c->d_v_cache && c->d_out,
              "diff_attn: null argument");
  ORN_REQUIRE(c->T >= 1 && c->H >= 1 && c->G >= 1 && c->H % c->G == 0 && c->G <= 65535 && c->dim >= 1 && c->vdim >= 1,
              "diff_attn: T=%d H=%d G=%d dim=%d vdim=%d", c->T, c->H, c->G, c->dim, c->vdim);
  ORN_REQUIRE(c->rope_dims >= 0 && c->rope_dims % 2 == 0 && c->rope_dims <= c->dim && (c->rope_dims == 0 || (c->d_cos && c->d_sin)),
              "diff_attn: %d rotated dimensions of %d", c->rope_dims, c->dim);
  ORN_REQUIRE(c->offset >= 0 && c->offset + c->T <= c->cap && (c->rope_dims == 0 || c->offset + c->T <= c->table_npos),
              "diff_attn: rows [%d, %d) in a cache of %d, tables of %d", c->offset, c->offset + c->T, c->cap, c->table_npos);
  ORN_REQUIRE(c->window >= 0 && c->keep_first >= 0, "diff_attn: window %d, kept %d", c->window, c->keep_first);
  DaArgs p{c->d_q, c->d_k, c->d_v, c->d_gate, c->d_cos, c->d_sin, c->rope_dims / 2, c->T, c->H, c->G, c->dim, c->vdim, c->offset,
           c->cap, c->window, c->keep_first, c->scale, c->lambda, c->diff, c->eps, c->d_k_cache, c->d_v_cache, c->d_q_rot, c->d_out};
  if (c->act == ORNITH_BF16 && c->T >= kPrefillRows && c->dim % 8 == 0 && c->vdim % 8 == 0 && c->dim <= 128 && c->vdim <= 256) {
    ORN_REQUIRE(c->d_q_rot, "diff_attn: %d rows need the buffer for the rotated queries", c->T);
    hipLaunchKernelGGL(diff_prep_kernel, dim3(p.T), dim3(NT), 0, ctx->stream, p);
    ORN_LAUNCH_CHECK("diff_prep_kernel");
    if (p.dim <= 32) launch_prefill<1>(ctx, p);
    else if (p.dim <= 64) launch_prefill<2>(ctx, p);
    else launch_prefill<4>(ctx, p);
    ORN_LAUNCH_CHECK("diff_prefill_kernel");
    return ORNITH_OK;
  }
  return c->act == ORNITH_F32 ? run_decode<float>(ctx, p) : run_decode<bf16_t>(ctx, p);
}
