// Latent attention (DeepSeek-AI, "DeepSeek-V2"): one low-rank row c and one turned key part a token, shared by
// all heads; a head's keys and values are linear maps of c. With a sliding window, a sink in the softmax's
// denominator and one output gate a head. The arithmetic is stated at ornith_latent_attn in ornith_hip.h.
//
// Decode widths (and 32-bit models): the key map goes into the query and the value map onto the result, so a
// cached row is read once for all heads and never expanded. Three launches: latent_query_kernel makes the
// queries uk^T q beside their turned part, and appends the call's rows to the cache; a decode kernel takes one
// block of a query's visible rows for a group of heads; latent_out_kernel joins a head's blocks, maps the
// result through uv and gates it. Everything between the bf16 operands is fp32. For bf16 rows of up to 576
// values the blocks run on the matrix cores (latent_mfma_kernel: heads are one side of both products; queries
// and softmax weights go in as two bf16 parts), others on the vector units (latent_decode_kernel). Blocks are
// counted along a query's own visible rows, so a row does not depend on what else is in the call.
//
// Prefill widths (bf16): the rows are appended, one GEMM makes keys and values of the rows in sight, and flash
// attention runs on the matrix cores, its keys the expanded part and the shared turned part side by side.
#include "act_device.h"
#include "mfma_device.h"
#include "rt.h"

namespace {

struct LaArgs {
  const void* q;
  const float* down;
  const bf16_t* down_norm;
  const bf16_t *uk, *uv;
  const float* gate;
  const bf16_t* sink;
  const float *cos_t, *sin_t;
  int T, H, dim, rot, vdim, rank, offset, cap, window;
  float scale, eps;
  void *c_cache, *r_cache, *out;
};

__device__ __forceinline__ int first_visible(const LaArgs& p, int pos) { return p.window > 0 ? max(0, pos - p.window + 1) : 0; }
// rows of a query's blocks: `unit`, or, where a workgroup can go on (a negative unit), twice as many until
// there are at most kMaxBlocks of them
constexpr int kMaxBlocks = 64;
__device__ __forceinline__ int block_rows(int nvis, int unit) {
  if (unit > 0) return unit;
  int kb = -unit;
  while (nvis > kMaxBlocks * kb) kb *= 2;
  return kb;
}
__device__ __forceinline__ float gate_at(const LaArgs& p, int t, int h) {
  return p.gate ? dm_sigmoid_f32(p.gate[(size_t)t * p.H + h]) : 1.0f;
}

// pair i of a turned part at position pos
__device__ __forceinline__ void turn_pair(const LaArgs& p, int pos, int i, float& u, float& v) {
  const size_t at = (size_t)pos * (p.rot / 2) + i;
  const float c = p.cos_t[at], s = p.sin_t[at], a = u, b = v;
  u = dm_fma(-b, s, a * c);
  v = dm_fma(a, s, b * c);
}

constexpr int NT = 256;

// One row of the cache, by a workgroup: the latent over its root mean square times its weight, the key
// part turned.
template <typename A>
__device__ __forceinline__ void append_row(const LaArgs& p, int t, float* red) {
  const int tid = threadIdx.x, pos = p.offset + t;
  const float* src = p.down + (size_t)t * (p.rank + p.rot);
  A* c = reinterpret_cast<A*>(p.c_cache) + (size_t)pos * p.rank;
  A* r = reinterpret_cast<A*>(p.r_cache) + (size_t)pos * p.rot;
  constexpr int PC = 4;
  float x[PC], a = 0.f;
#pragma unroll
  for (int i = 0; i < PC; ++i) {
    const int d = tid + NT * i;
    x[i] = d < p.rank ? src[d] : 0.f;
    a = dm_fma(x[i], x[i], a);
  }
  for (int d = tid + NT * PC; d < p.rank; d += NT) a = dm_fma(src[d], src[d], a);
  for (int i = tid; i < p.rot / 2; i += NT) {
    float u = src[p.rank + 2 * i], v = src[p.rank + 2 * i + 1];
    turn_pair(p, pos, i, u, v);
    r[2 * i] = act_of<A>(u);
    r[2 * i + 1] = act_of<A>(v);
  }
  a = dm_wave_sum<64>(a);
  __syncthreads();
  if ((tid & 63) == 0) red[tid >> 6] = a;
  __syncthreads();
  const float inv = dm_rsqrt((((red[0] + red[1]) + red[2]) + red[3]) / (float)p.rank + p.eps);
#pragma unroll
  for (int i = 0; i < PC; ++i) {
    const int d = tid + NT * i;
    if (d < p.rank) c[d] = act_of<A>((x[i] * inv) * dm_bf2f(p.down_norm[d]));
  }
  for (int d = tid + NT * PC; d < p.rank; d += NT) c[d] = act_of<A>((src[d] * inv) * dm_bf2f(p.down_norm[d]));
}

// ---- decode widths ---------------------------------------------------------------------
constexpr int QC = 128, DG = NT / 16;  // latent columns of a query workgroup; its groups of head dimensions

// Queries over the cached rows, [T][H][rank + rot, padded with zeros to `stride`], scaled: fp32 or as two
// bf16 parts.
struct MappedQ {
  float* f;
  bf16_t *hi, *lo;
  int stride;
  __device__ __forceinline__ void put(size_t at, float v) const {
    if (f) {
      f[at] = v;
    } else {
      const bf16_t h = dm_f2bf(v);
      hi[at] = h;
      lo[at] = dm_f2bf(v - dm_bf2f(h));
    }
  }
};

// grid (column tiles, H + 1, row groups). The last grid row appends.
template <typename A, int MR, bool VEC>
__global__ __launch_bounds__(NT) void latent_query_kernel(LaArgs p, MappedQ qs) {
  extern __shared__ __attribute__((aligned(16))) char lds_raw[];
  float* red = reinterpret_cast<float*>(lds_raw);  // [DG][MR][QC]
  float* xq = red + DG * MR * QC;                  // [MR][dim]
  const int tid = threadIdx.x, h = blockIdx.y, m0 = blockIdx.z * MR, n = min(MR, p.T - m0);
  if (h == p.H) {
    if (blockIdx.x == 0 && p.down)
      for (int m = 0; m < n; ++m) append_row<A>(p, m0 + m, red);
    return;  // (the whole workgroup)
  }
  const int qd = p.dim + p.rot, QS = qs.stride;
  const int cg = tid & 15, dg = tid >> 4, r0 = blockIdx.x * QC + 8 * cg;
  const bf16_t* w = p.uk + (size_t)h * p.dim * p.rank + r0;
  const int in = min(8, p.rank - r0);  // columns of this thread that exist
  auto piece = [&](int d) -> uint4 {
    if (in <= 0 || d >= p.dim) return make_uint4(0, 0, 0, 0);
    const bf16_t* s = w + (size_t)d * p.rank;
    if constexpr (VEC) return *reinterpret_cast<const uint4*>(s);
    uint32_t e[8];
#pragma unroll
    for (int i = 0; i < 8; ++i) e[i] = i < in ? s[i] : 0;
    return make_uint4(e[0] | e[1] << 16, e[2] | e[3] << 16, e[4] | e[5] << 16, e[6] | e[7] << 16);
  };
  constexpr int U = 8;
  uint4 cur[U];
#pragma unroll
  for (int u = 0; u < U; ++u) cur[u] = piece(dg + DG * u);
  const A* q = reinterpret_cast<const A*>(p.q);
  for (int i = tid; i < MR * p.dim; i += NT) {
    const int m = i / p.dim, d = i % p.dim;
    xq[i] = m < n ? act_f(q[((size_t)(m0 + m) * p.H + h) * qd + d]) : 0.f;
  }
  if (blockIdx.x == 0)
    for (int i = tid; i < n * (p.rot / 2); i += NT) {
      const int m = i / (p.rot / 2), e = i % (p.rot / 2);
      const A* s = q + ((size_t)(m0 + m) * p.H + h) * qd + p.dim + 2 * e;
      float u = act_f(s[0]), v = act_f(s[1]);
      turn_pair(p, p.offset + m0 + m, e, u, v);
      const size_t at = ((size_t)(m0 + m) * p.H + h) * QS + p.rank + 2 * e;
      qs.put(at, u * p.scale);
      qs.put(at + 1, v * p.scale);
    }
  const int pad = QS - p.rank - p.rot;
  if (blockIdx.x == 0)
    for (int i = tid; i < n * pad; i += NT) qs.put(((size_t)(m0 + i / pad) * p.H + h) * QS + p.rank + p.rot + i % pad, 0.f);
  __syncthreads();
  float acc[MR][8];
#pragma unroll
  for (int m = 0; m < MR; ++m)
#pragma unroll
    for (int e = 0; e < 8; ++e) acc[m][e] = 0.f;
  for (int d0 = dg; d0 < p.dim; d0 += DG * U) {
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int d = d0 + DG * u;
      const uint4 c = cur[u];
      cur[u] = piece(d + DG * U);
      if (d >= p.dim) continue;
      const float wv[8] = {dm_bf2f_lo(c.x), dm_bf2f_hi(c.x), dm_bf2f_lo(c.y), dm_bf2f_hi(c.y),
                           dm_bf2f_lo(c.z), dm_bf2f_hi(c.z), dm_bf2f_lo(c.w), dm_bf2f_hi(c.w)};
#pragma unroll
      for (int m = 0; m < MR; ++m) {
        const float x = xq[m * p.dim + d];
#pragma unroll
        for (int e = 0; e < 8; ++e) acc[m][e] = dm_fma(x, wv[e], acc[m][e]);
      }
    }
  }
#pragma unroll
  for (int m = 0; m < MR; ++m)
#pragma unroll
    for (int e = 0; e < 8; ++e) red[(dg * MR + m) * QC + 8 * cg + e] = acc[m][e];
  __syncthreads();
  for (int i = tid; i < n * QC; i += NT) {
    const int m = i / QC, c = i % QC, r = blockIdx.x * QC + c;
    if (r >= p.rank) continue;
    float a = 0.f;
#pragma unroll
    for (int g = 0; g < DG; ++g) a += red[(g * MR + m) * QC + c];
    qs.put(((size_t)(m0 + m) * p.H + h) * QS + r, a * p.scale);
  }
}

// grid (blocks, head groups, rows): KB rows of a query's visible ones against HG heads. part: f32
// [rows][H][blocks][rank], ml: [rows][H][blocks][2]. A score is summed by NT / (KB HG) neighbouring lanes.
template <typename A, bool VEC>
__global__ __launch_bounds__(NT) void latent_decode_kernel(LaArgs p, const float* qs, int KB, int HG, int t_base, float* part,
                                                           float* ml) {
  extern __shared__ __attribute__((aligned(16))) char lds_raw[];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int t = t_base + blockIdx.z, pos = p.offset + t, lo = first_visible(p, pos), nvis = pos - lo + 1;
  const int u0 = blockIdx.x * KB;
  if (u0 >= nvis) return;  // (every thread of the workgroup)
  const int nk = min(KB, nvis - u0), blocks = gridDim.x;
  const int h0 = blockIdx.y * HG, nh = min(HG, p.H - h0);
  const int QS = p.rank + p.rot, q4 = (QS + 3) & ~3, cst = ((QS + 7) & ~7) + 16 / (int)sizeof(A);
  float* xq = reinterpret_cast<float*>(lds_raw);  // [HG][q4]
  float* sc = xq + HG * q4;                       // [HG][KB]
  A* cs = reinterpret_cast<A*>(sc + HG * KB);     // [KB][cst]: latent, turned part
  const A* cc = reinterpret_cast<const A*>(p.c_cache) + (size_t)(lo + u0) * p.rank;
  const A* rc = reinterpret_cast<const A*>(p.r_cache) + (size_t)(lo + u0) * p.rot;
  const float* qsrc = qs + ((size_t)t * p.H + h0) * QS;
  if constexpr (VEC) {
    constexpr int E = 16 / (int)sizeof(A), B = 8;
    const int cch = p.rank / E, rch = p.rot / E, per = cch + rch, n = nk * per;
    auto load = [&](int i) {
      const int r = i / per, c = i % per;
      return c < cch ? *reinterpret_cast<const uint4*>(cc + (size_t)r * p.rank + c * E)
                     : *reinterpret_cast<const uint4*>(rc + (size_t)r * p.rot + (c - cch) * E);
    };
    // asked for before any of it is waited for
    uint4 x[B];
#pragma unroll
    for (int b = 0; b < B; ++b)
      if (tid + NT * b < n) x[b] = load(tid + NT * b);
    for (int i = tid; i < nh * QS / 4; i += NT) reinterpret_cast<float4*>(xq)[i] = reinterpret_cast<const float4*>(qsrc)[i];
#pragma unroll
    for (int b = 0; b < B; ++b) {
      const int i = tid + NT * b;
      if (i < n) *reinterpret_cast<uint4*>(&cs[(i / per) * cst + (i % per) * E]) = x[b];
    }
    for (int i = tid + NT * B; i < n; i += NT) *reinterpret_cast<uint4*>(&cs[(i / per) * cst + (i % per) * E]) = load(i);
  } else {
    for (int i = tid; i < nk * QS; i += NT) {
      const int r = i / QS, c = i % QS;
      cs[r * cst + c] = c < p.rank ? cc[(size_t)r * p.rank + c] : rc[(size_t)r * p.rot + c - p.rank];
    }
    for (int i = tid; i < nh * QS; i += NT) xq[(i / QS) * q4 + i % QS] = qsrc[i];
  }
  __syncthreads();
  {
    const int P = NT / (KB * HG), part_i = tid % P, key = (tid / P) % KB, hh = tid / (P * KB);
    float s = 0.f;
    if (key < nk && hh < nh) {
      const A* kr = cs + key * cst;
      const float* qr = xq + hh * q4;
      if constexpr (VEC) {
#pragma unroll 4
        for (int c = 8 * part_i; c < QS; c += 8 * P) {
          float kv[8], qv[8];
          act_load<8>(kr + c, kv);
          act_load<8>(qr + c, qv);
#pragma unroll
          for (int e = 0; e < 8; ++e) s = dm_fma(kv[e], qv[e], s);
        }
      } else {
        for (int c = part_i; c < QS; c += P) s = dm_fma(act_f(kr[c]), qr[c], s);
      }
    }
    for (int o = P / 2; o > 0; o >>= 1) s += __shfl_xor(s, o);
    if (part_i == 0) sc[hh * KB + key] = key < nk && hh < nh ? s : -DM_INF;
  }
  __syncthreads();
  // a head's maximum, exponentials and sum: one wavefront a head
  for (int r = wave; r < nh; r += NT / 64) {
    const float s = lane < KB ? sc[r * KB + lane] : -DM_INF;
    const float m = dm_wave_max<64>(s);
    const float e = s == -DM_INF ? 0.f : dm_exp(s - m);
    const float l = dm_wave_sum<64>(e);
    if (lane < KB) sc[r * KB + lane] = e;
    if (lane == 0) {
      float* d = ml + (((size_t)blockIdx.z * p.H + h0 + r) * blocks + blockIdx.x) * 2;
      d[0] = m;
      d[1] = l;
    }
  }
  __syncthreads();
  constexpr int W = VEC ? 4 : 1;
  const int cols = p.rank / W;
  for (int i = tid; i < nh * cols; i += NT) {
    const int r = i / cols, c = (i % cols) * W;
    float o[W];
#pragma unroll
    for (int e = 0; e < W; ++e) o[e] = 0.f;
    const float* pr = sc + r * KB;
#pragma unroll 8
    for (int key = 0; key < nk; ++key) {
      const float w = pr[key];
      if constexpr (VEC) {
        float vv[4];
        act_load<4>(&cs[key * cst + c], vv);
#pragma unroll
        for (int e = 0; e < W; ++e) o[e] = dm_fma(w, vv[e], o[e]);
      } else {
        o[0] = dm_fma(w, act_f(cs[key * cst + c]), o[0]);
      }
    }
    float* d = part + (((size_t)blockIdx.z * p.H + h0 + r) * blocks + blockIdx.x) * p.rank + c;
    if constexpr (VEC) {
      act_store4(d, o);
    } else {
      d[0] = o[0];
    }
  }
}

// grid (value tiles, H, rows): the blocks of a query joined with weights e^(m_b - M), groups of threads taking
// every G-th block, then VB values of the head, a wavefront VB / 8 of them.
constexpr int VB = 64, ONT = 512;
template <typename A, bool VEC>
__global__ __launch_bounds__(ONT) void latent_out_kernel(LaArgs p, int unit, int t_base, int stride, const float* part, const float* ml) {
  extern __shared__ __attribute__((aligned(16))) char lds_raw[];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int h = blockIdx.y, t = t_base + blockIdx.z, pos = p.offset + t;
  const int nvis = pos - first_visible(p, pos) + 1, KB = block_rows(nvis, unit), nb = (nvis + KB - 1) / KB;
  const int rp = (p.rank + 7) & ~7;
  float* ol = reinterpret_cast<float*>(lds_raw);  // [rank rounded up to 8]
  float* wb = ol + rp;                            // [stride rounded up to 4]
  float* red = wb + ((stride + 3) & ~3);          // [G][rank]
  const size_t base = ((size_t)blockIdx.z * p.H + h) * stride;
  // this wavefront's weights, asked for ahead
  constexpr int VR = VB / (ONT / 64);
  const int v0 = blockIdx.x * VB + wave * VR;
  const bf16_t* w = p.uv + ((size_t)h * p.vdim + v0) * p.rank;
  uint4 first[VR];
  if constexpr (VEC) {
#pragma unroll
    for (int r = 0; r < VR; ++r)
      if (v0 + r < p.vdim && 8 * lane < p.rank) first[r] = *reinterpret_cast<const uint4*>(w + (size_t)r * p.rank + 8 * lane);
  }
  // four columns a thread, and the first blocks of its group, asked for before the weights are made
  constexpr int W = VEC ? 4 : 1, U = 8;
  const int cols = p.rank / W, G = max(1, ONT / cols), g = tid / cols, c0 = tid % cols;
  const float* src = part + base * p.rank;
  float x[U][W];
  auto fetch = [&](int b0, int c) {
#pragma unroll
    for (int u = 0; u < U; ++u) {
      const int b = min(b0 + G * u, nb - 1);
      if constexpr (VEC) act_load<4>(src + (size_t)b * p.rank + 4 * c, x[u]);
      else x[u][0] = src[(size_t)b * p.rank + c];
    }
  };
  if (g < G) fetch(g, c0);
  if (wave == 0) {
    const float sink = p.sink ? dm_bf2f(p.sink[h]) : -DM_INF;
    const float* mr = ml + base * 2;
    float M = sink;
    for (int b = lane; b < nb; b += 64) M = __builtin_fmaxf(M, mr[2 * b]);
    M = dm_wave_max<64>(M);
    float L = 0.f;
    for (int b = lane; b < nb; b += 64) {
      const float e = dm_exp(mr[2 * b] - M);
      wb[b] = e;
      L = dm_fma(e, mr[2 * b + 1], L);
    }
    L = dm_wave_sum<64>(L);
    if (p.sink) L += dm_exp(sink - M);
    for (int b = lane; b < nb; b += 64) wb[b] = wb[b] / L;
  }
  __syncthreads();
  for (int c = c0; c < cols; c += ONT) {  // (one round unless a row is longer than the workgroup)
    if (g < G) {
      float o[W];
#pragma unroll
      for (int e = 0; e < W; ++e) o[e] = 0.f;
      if (c != c0) fetch(g, c);
      for (int b0 = g; b0 < nb; b0 += G * U) {
#pragma unroll
        for (int u = 0; u < U; ++u) {
          const float wt = b0 + G * u < nb ? wb[b0 + G * u] : 0.f;
#pragma unroll
          for (int e = 0; e < W; ++e) o[e] = b0 + G * u < nb ? dm_fma(wt, x[u][e], o[e]) : o[e];
        }
        if (b0 + G * U < nb) fetch(b0 + G * U, c);
      }
#pragma unroll
      for (int e = 0; e < W; ++e) red[g * p.rank + W * c + e] = o[e];
    }
  }
  __syncthreads();
  for (int c = tid; c < rp; c += ONT) {
    float o = 0.f;
    if (c < p.rank)
      for (int i = 0; i < G; ++i) o += red[i * p.rank + c];
    ol[c] = o;
  }
  __syncthreads();
  const float gt = gate_at(p, t, h);
  A* dst = reinterpret_cast<A*>(p.out) + ((size_t)t * p.H + h) * p.vdim;
  float a[VR];
#pragma unroll
  for (int r = 0; r < VR; ++r) a[r] = 0.f;
  if constexpr (VEC) {
    for (int c = 8 * lane; c < p.rank; c += 512) {
      float ov[8];
      act_load<8>(ol + c, ov);
#pragma unroll
      for (int r = 0; r < VR; ++r) {
        if (v0 + r >= p.vdim) continue;
        const uint4 y = c == 8 * lane ? first[r] : *reinterpret_cast<const uint4*>(w + (size_t)r * p.rank + c);
        const float wv[8] = {dm_bf2f_lo(y.x), dm_bf2f_hi(y.x), dm_bf2f_lo(y.y), dm_bf2f_hi(y.y),
                             dm_bf2f_lo(y.z), dm_bf2f_hi(y.z), dm_bf2f_lo(y.w), dm_bf2f_hi(y.w)};
#pragma unroll
        for (int e = 0; e < 8; ++e) a[r] = dm_fma(wv[e], ov[e], a[r]);
      }
    }
  } else {
#pragma unroll
    for (int r = 0; r < VR; ++r)
      if (v0 + r < p.vdim)
        for (int c = lane; c < p.rank; c += 64) a[r] = dm_fma(dm_bf2f(w[(size_t)r * p.rank + c]), ol[c], a[r]);
  }
#pragma unroll
  for (int r = 0; r < VR; ++r) a[r] = dm_wave_sum<64>(a[r]);
#pragma unroll
  for (int r = 0; r < VR; ++r)
    if (lane == r && v0 + r < p.vdim) dst[v0 + r] = act_of<A>(a[r] * gt);
}

typedef __bf16 l_bf16x8 __attribute__((ext_vector_type(8)));
typedef float l_f32x4 __attribute__((ext_vector_type(4)));
typedef uint32_t l_u32x4 __attribute__((ext_vector_type(4)));

// The same blocks on the matrix cores, 32 rows a step: grid (blocks, groups of 16 heads, rows). Scores run as
// S^T = C Q^T: wavefront (key half, channel half) takes sixteen rows of the step over half of their channels,
// straight from memory; softmax by sixteen threads a head; O^T += C^T P^T with the rows turned in LDS, a
// wavefront every fourth tile of sixteen columns. NS: 32-channel steps of a wavefront, CT: its column tiles;
// rows of at most 64 NS values (queries padded to that with zeros), latents of at most 64 CT. Loads past a
// row's end fetch its last piece again: they meet zeros, or columns nobody stores. The loop's body is the same
// from the first step on (weights start at e^-inf) and not unrolled: at these widths a launch waits for its
// instructions as much as for its data.
constexpr int MK = 32, MV = MK + 8, MH = 16;
template <int NS, int CT>
__global__ __launch_bounds__(NT, 1) void latent_mfma_kernel(LaArgs p, const bf16_t* q_hi, const bf16_t* q_lo, int t_base, float* part,
                                                            float* ml) {
  constexpr int TPH = NT / MH, KPT = MK / TPH, VI = (CT + 1) / 2;  // threads a head, keys of such a thread
  static_assert(KPT == 2, "a thread's weights are a pair");
  __shared__ __attribute__((aligned(16))) bf16_t Vt[VI * 128][MV];
  __shared__ __attribute__((aligned(16))) float sp[2][MH][MK + 4];
  __shared__ __attribute__((aligned(16))) bf16_t Ph[MH][MV], Pl[MH][MV];
  __shared__ float al[MH];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, l16 = lane & 15, lg = lane >> 4;
  const int t = t_base + blockIdx.z, pos = p.offset + t, lo = first_visible(p, pos), nvis = pos - lo + 1;
  const int KB = block_rows(nvis, -MK), u0 = blockIdx.x * KB;
  if (u0 >= nvis) return;  // (every thread of the workgroup)
  const int u1 = min(nvis, u0 + KB), h0 = blockIdx.y * MH, QS = p.rank + p.rot;
  const int kt = wave & 1, s0 = (wave >> 1) * NS;
  const bf16_t* cc = reinterpret_cast<const bf16_t*>(p.c_cache);
  const bf16_t* rc = reinterpret_cast<const bf16_t*>(p.r_cache);
  // rows as score operands, and pairs of rows to be turned
  l_bf16x8 kf[NS];
  l_u32x4 vr[VI][2];
  const int pair = (tid >> 2) & 15, oct0 = (tid & 3) + 4 * (tid >> 6);
  auto fetch = [&](int u) {
    const size_t row = lo + min(u + 16 * kt + l16, nvis - 1);
    const bf16_t *ck = cc + row * p.rank, *rk = rc + row * p.rot - p.rank;
#pragma unroll
    for (int i = 0; i < NS; ++i) {
      const int d = min(32 * (s0 + i) + 8 * lg, QS - 8);
      kf[i] = __builtin_bit_cast(l_bf16x8, *reinterpret_cast<const l_u32x4*>((d < p.rank ? ck : rk) + d));
    }
#pragma unroll
    for (int b = 0; b < 2; ++b) {
      const bf16_t* cv = cc + (size_t)(lo + min(u + 2 * pair + b, nvis - 1)) * p.rank;
#pragma unroll
      for (int i = 0; i < VI; ++i) vr[i][b] = *reinterpret_cast<const l_u32x4*>(cv + min(8 * (oct0 + 16 * i), p.rank - 8));
    }
  };
  fetch(u0);
  l_bf16x8 qh[NS], ql[NS];
  const size_t q_at = ((size_t)t * p.H + min(h0 + l16, p.H - 1)) * (64 * NS) + 32 * s0 + 8 * lg;
#pragma unroll
  for (int i = 0; i < NS; ++i) {
    qh[i] = *reinterpret_cast<const l_bf16x8*>(q_hi + q_at + 32 * i);
    ql[i] = *reinterpret_cast<const l_bf16x8*>(q_lo + q_at + 32 * i);
  }
  l_f32x4 acc[CT];
#pragma unroll
  for (int c = 0; c < CT; ++c) acc[c] = l_f32x4{0.f, 0.f, 0.f, 0.f};
  const int hh = tid / TPH, sub = tid % TPH;  // a head's softmax
  float m = -DM_INF, l = 0.f;
#pragma clang loop unroll(disable)
  for (int u = u0; u < u1; u += MK) {
    l_f32x4 sc[2] = {l_f32x4{0.f, 0.f, 0.f, 0.f}, l_f32x4{0.f, 0.f, 0.f, 0.f}};
#pragma unroll
    for (int i = 0; i < NS; ++i) {
      sc[0] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf[i], qh[i], sc[0], 0, 0, 0);
      sc[1] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf[i], ql[i], sc[1], 0, 0, 0);
    }
    __syncthreads();  // the step before is done with LDS
    *reinterpret_cast<l_f32x4*>(&sp[wave >> 1][l16][16 * kt + 4 * lg]) = sc[0] + sc[1];
#pragma unroll
    for (int i = 0; i < VI; ++i) {
      bf16_t* v = &Vt[8 * (oct0 + 16 * i)][2 * pair];
#pragma unroll
      for (int w = 0; w < 4; ++w) {
        *reinterpret_cast<uint32_t*>(v + 2 * w * MV) = __builtin_amdgcn_perm(vr[i][1][w], vr[i][0][w], 0x05040100u);
        *reinterpret_cast<uint32_t*>(v + (2 * w + 1) * MV) = __builtin_amdgcn_perm(vr[i][1][w], vr[i][0][w], 0x07060302u);
      }
    }
    if (u + MK < u1) fetch(u + MK);
    __syncthreads();
    {
      const float2 a = *reinterpret_cast<const float2*>(&sp[0][hh][KPT * sub]), b = *reinterpret_cast<const float2*>(&sp[1][hh][KPT * sub]);
      const float x = u + KPT * sub < u1 ? a.x + b.x : -DM_INF, y = u + KPT * sub + 1 < u1 ? a.y + b.y : -DM_INF;
      const float mn = __builtin_fmaxf(m, dm_wave_max<TPH>(__builtin_fmaxf(x, y)));
      const float alpha = dm_exp(m - mn), ex = dm_exp(x - mn), ey = dm_exp(y - mn);
      l = dm_fma(l, alpha, dm_wave_sum<TPH>(ex + ey));
      m = mn;
      uint32_t hi, lo2;
      split2(ex, ey, hi, lo2);
      *reinterpret_cast<uint32_t*>(&Ph[hh][KPT * sub]) = hi;
      *reinterpret_cast<uint32_t*>(&Pl[hh][KPT * sub]) = lo2;
      if (sub == 0) al[hh] = alpha;
    }
    __syncthreads();
    const l_bf16x8 ph = *reinterpret_cast<const l_bf16x8*>(&Ph[l16][8 * lg]), pl = *reinterpret_cast<const l_bf16x8*>(&Pl[l16][8 * lg]);
    const float x = al[l16];
#pragma unroll
    for (int c = 0; c < CT; ++c) {
      const l_bf16x8 vf = *reinterpret_cast<const l_bf16x8*>(&Vt[16 * (wave + 4 * c) + l16][8 * lg]);
      acc[c] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf, ph, acc[c] * x, 0, 0, 0);
      acc[c] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf, pl, acc[c], 0, 0, 0);
    }
  }
  const int blocks = gridDim.x, h = h0 + l16;
  if (h < p.H) {
    float* dst = part + (((size_t)blockIdx.z * p.H + h) * blocks + blockIdx.x) * p.rank;
#pragma unroll
    for (int c = 0; c < CT; ++c) {
      const int col = 16 * (wave + 4 * c) + 4 * lg;
      if (col < p.rank) *reinterpret_cast<l_f32x4*>(dst + col) = acc[c];
    }
  }
  if (sub == 0 && h0 + hh < p.H) {
    float* d = ml + (((size_t)blockIdx.z * p.H + h0 + hh) * blocks + blockIdx.x) * 2;
    d[0] = m;
    d[1] = l;
  }
}

template <typename A, int MR>
int launch_query(ornith_ctx* ctx, const LaArgs& p, bool vec, const MappedQ& qs) {
  const size_t lds = (size_t)(DG * MR * QC + MR * p.dim) * 4;
  const dim3 grid((p.rank + QC - 1) / QC, p.H + (p.down ? 1 : 0), (p.T + MR - 1) / MR);
  ORN_REQUIRE(lds <= 65536, "latent_attn: heads of %d dimensions", p.dim);
  if (vec) hipLaunchKernelGGL((latent_query_kernel<A, MR, true>), grid, dim3(NT), lds, ctx->stream, p, qs);
  else hipLaunchKernelGGL((latent_query_kernel<A, MR, false>), grid, dim3(NT), lds, ctx->stream, p, qs);
  ORN_LAUNCH_CHECK("latent_query_kernel");
  return ORNITH_OK;
}

template <int NS, int CT>
void launch_mfma(ornith_ctx* ctx, const LaArgs& p, const MappedQ& q, int blocks, int t, int n, float* part, float* ml) {
  hipLaunchKernelGGL((latent_mfma_kernel<NS, CT>), dim3(blocks, (p.H + MH - 1) / MH, n), dim3(NT), 0, ctx->stream, p, q.hi, q.lo, t,
                     part, ml);
}

template <typename A>
int run_decode(ornith_ctx* ctx, const LaArgs& p) {
  const bool vec = p.rank % 8 == 0 && p.rot % 8 == 0;
  const int QS = p.rank + p.rot, NS = (QS + 63) / 64;
  const bool mfma = sizeof(A) == 2 && vec && p.rank <= 512 && NS <= 9;
  const size_t q4 = (QS + 3) & ~3, cst = ((QS + 7) & ~7) + 16 / sizeof(A);
  int HG = 1;
  while (HG < 4 && HG < p.H) HG *= 2;
  int KB = 32;
  auto lds_of = [&]() { return (size_t)HG * (q4 + KB) * 4 + KB * cst * sizeof(A); };
  while (lds_of() > 65536 && KB > 8) KB /= 2;
  while (lds_of() > 65536 && HG > 1) HG /= 2;
  const size_t lds = lds_of();
  if (!mfma) {
    ORN_REQUIRE(lds <= 160 * 1024, "latent_attn: rows of %d values do not fit a compute unit's local memory", QS);
    if (lds > 65536) {
      ORN_HIP(hipFuncSetAttribute((const void*)latent_decode_kernel<A, true>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds));
      ORN_HIP(hipFuncSetAttribute((const void*)latent_decode_kernel<A, false>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds));
    }
  }
  const int last = p.offset + p.T - 1;
  const int most = p.window > 0 && p.window < last + 1 ? p.window : last + 1;
  const int unit = mfma ? -MK : KB, cut = (most + (mfma ? MK : KB) - 1) / (mfma ? MK : KB);
  const int blocks = mfma && cut > kMaxBlocks ? kMaxBlocks : cut;  // of the query that has the most
  // rows in groups whose partial results stay below 256 MB
  const size_t per = (size_t)p.H * blocks * (p.rank + 2) * 4, fit = (size_t(256) << 20) / per;
  int group = p.T < 32768 ? p.T : 32768;
  if ((size_t)group > fit) group = fit < 1 ? 1 : (int)fit;
  MappedQ qs{};
  qs.stride = mfma ? 64 * (NS <= 3 ? 3 : NS <= 6 ? 6 : 9) : QS;
  const size_t nq = (size_t)p.T * p.H * qs.stride;
  void* base = nullptr;
  int rc = ornith_scratch(ctx, nq * 4 + per * group + 8 * 256, &base);
  if (rc) return rc;
  ScratchCursor sc(base);
  if (mfma) {
    qs.hi = sc.take<bf16_t>(nq);
    qs.lo = sc.take<bf16_t>(nq);
  } else {
    qs.f = sc.take<float>(nq);
  }
  float* part = sc.take<float>((size_t)group * p.H * blocks * p.rank);
  float* ml = sc.take<float>((size_t)group * p.H * blocks * 2);
  rc = p.T == 1 ? launch_query<A, 1>(ctx, p, vec, qs) : p.T == 2 ? launch_query<A, 2>(ctx, p, vec, qs) : launch_query<A, 4>(ctx, p, vec, qs);
  if (rc) return rc;
  const int cols = vec ? p.rank / 4 : p.rank, G = cols < ONT ? ONT / cols : 1;
  const size_t olds = (size_t)(((p.rank + 7) & ~7) + ((blocks + 3) & ~3) + G * p.rank) * 4;
  ORN_REQUIRE(olds <= 65536, "latent_attn: %d blocks of rows in sight, rank %d", blocks, p.rank);
  for (int t = 0; t < p.T; t += group) {
    const int n = p.T - t < group ? p.T - t : group;
    const dim3 grid(blocks, (p.H + HG - 1) / HG, n), ogrid((p.vdim + VB - 1) / VB, p.H, n);
    if (mfma) {
      if (NS <= 3) launch_mfma<3, 3>(ctx, p, qs, blocks, t, n, part, ml);
      else if (NS <= 6) launch_mfma<6, 6>(ctx, p, qs, blocks, t, n, part, ml);
      else launch_mfma<9, 8>(ctx, p, qs, blocks, t, n, part, ml);
    } else if (vec) {
      hipLaunchKernelGGL((latent_decode_kernel<A, true>), grid, dim3(NT), lds, ctx->stream, p, qs.f, KB, HG, t, part, ml);
    } else {
      hipLaunchKernelGGL((latent_decode_kernel<A, false>), grid, dim3(NT), lds, ctx->stream, p, qs.f, KB, HG, t, part, ml);
    }
    ORN_LAUNCH_CHECK("latent attention over a block");
    if (vec) hipLaunchKernelGGL((latent_out_kernel<A, true>), ogrid, dim3(ONT), olds, ctx->stream, p, unit, t, blocks, part, ml);
    else hipLaunchKernelGGL((latent_out_kernel<A, false>), ogrid, dim3(ONT), olds, ctx->stream, p, unit, t, blocks, part, ml);
    ORN_LAUNCH_CHECK("latent_out_kernel");
  }
  return ORNITH_OK;
}

// ---- prefill widths ----------------------------------------------------------------------
__global__ __launch_bounds__(NT) void latent_append_kernel(LaArgs p) {
  __shared__ float red[4];
  append_row<bf16_t>(p, blockIdx.x, red);
}

constexpr int BKV = 64, LV = BKV + 8;

// keys [rows][H][dim] and values [rows][H][vdim] of the cached rows from `base` (a multiple of BKV) on
struct Expanded {
  const bf16_t *k, *v;
  int base;
};

// One workgroup: 64 S query rows of one head, S groups of sixteen a wavefront. Both products run transposed
// (S^T = K Q^T, O^T += V^T P^T): a lane owns a query from the scores to the output, the weights never leave
// the registers, and a key or value fragment read from LDS serves every group. The weights go to the matrix
// cores as two bf16 parts, so they count as 32-bit numbers. A key row in LDS is its expanded part, padded to
// 32 channels, then the shared turned part. KD: 32-channel steps of a key; VT: 16-channel tiles of the values.
template <int KD, int VT, int S>
__global__ __launch_bounds__(256, VT <= 8 && KD <= 4 ? 2 : 1) void latent_prefill_kernel(LaArgs p, Expanded x) {
  constexpr int DP = KD * 32, LK = DP + 8, BQ = 64 * S;
  __shared__ __attribute__((aligned(16))) bf16_t Ks[BKV][LK];
  __shared__ __attribute__((aligned(16))) bf16_t Vt[VT * 16][LV];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, l16 = lane & 15, lg = lane >> 4;
  // the last rows of a call see the most: they start first
  const int qt = gridDim.y - 1 - blockIdx.y, h = blockIdx.x;
  const int t0 = qt * BQ, first = p.offset + t0, last = p.offset + min(t0 + BQ, p.T) - 1;
  const int dimp = (p.dim + 31) & ~31;  // where the turned part starts
  int tq[S], pos[S];
  l_bf16x8 qf[S][KD];
#pragma unroll
  for (int s = 0; s < S; ++s) {
    tq[s] = t0 + (wave * S + s) * 16 + l16;
    const int tc = min(tq[s], p.T - 1);
    pos[s] = p.offset + tc;
    const bf16_t* row = reinterpret_cast<const bf16_t*>(p.q) + ((size_t)tc * p.H + h) * (p.dim + p.rot);
#pragma unroll
    for (int kk = 0; kk < KD; ++kk) {
      const int d = 32 * kk + 8 * lg, e = d - dimp;
      l_u32x4 w = {0, 0, 0, 0};
      if (d < p.dim) {
        w = *reinterpret_cast<const l_u32x4*>(row + d);
      } else if (e >= 0 && e < p.rot) {
        w = *reinterpret_cast<const l_u32x4*>(row + p.dim + e);
#pragma unroll
        for (int i = 0; i < 4; ++i) {
          float a = dm_bf2f_lo(w[i]), b = dm_bf2f_hi(w[i]);
          turn_pair(p, pos[s], e / 2 + i, a, b);
          w[i] = dm_f2bf2(a, b);
        }
      }
      if (p.scale < 0.f) w ^= 0x80008000u;  // the scale's sign, so that a row's largest score is its largest product
      qf[s][kk] = __builtin_bit_cast(l_bf16x8, w);
    }
  }
  const float s2 = __builtin_fmaxf(__builtin_fabsf(p.scale) * 1.44269504088896341f, 1e-30f);
  // the sink is one more score, counted once (by one of the four lanes that share a query)
  const float sink = p.sink ? dm_bf2f(p.sink[h]) * 1.44269504088896341f : -DM_INF;
  l_f32x4 acc[S][VT];
  float mx[S], sum[S];
#pragma unroll
  for (int s = 0; s < S; ++s) {
    mx[s] = sink;
    sum[s] = p.sink && lg == 0 ? 1.f : 0.f;
#pragma unroll
    for (int v = 0; v < VT; ++v) acc[s][v] = l_f32x4{0.f, 0.f, 0.f, 0.f};
  }
  const int lo = first_visible(p, first), wb0 = lo / BKV, nblocks = last / BKV - wb0 + 1;
  // this thread's pieces of a key block: 16 bytes of a key row each, and pairs of value rows, turned on
  // their way into LDS; the next block's are asked for before this one is worked on. Value piece e: four
  // neighbouring lanes read 64 bytes of a row, and the sixteen row pairs of a wavefront keep its LDS
  // writes two to a bank.
  constexpr int KI = KD, VI = VT / 4;
  l_u32x4 kreg[KI], vreg[VI][2];
  int krow[KI], kcol[KI], kstr[KI], vrow[VI], vcol[VI];
  bool kin[KI], krot[KI], vin[VI];
#pragma unroll
  for (int i = 0; i < KI; ++i) {
    const int e = tid + 256 * i, d = 8 * (e % (4 * KD));
    krow[i] = e / (4 * KD);
    krot[i] = d >= dimp;
    kin[i] = krot[i] ? d - dimp < p.rot : d < p.dim;
    kcol[i] = !kin[i] ? 0 : krot[i] ? d - dimp : d;
    kstr[i] = krot[i] ? p.rot : p.H * p.dim;
  }
#pragma unroll
  for (int i = 0; i < VI; ++i) {
    const int e = tid + 256 * i, d = 8 * ((e & 3) + 4 * (e >> 7));
    vrow[i] = 2 * ((e >> 2) & 31);
    vin[i] = d < p.vdim;
    vcol[i] = vin[i] ? d : 0;
  }
  const bf16_t* kx = x.k + (size_t)h * p.dim;
  const bf16_t* vx = x.v + (size_t)h * p.vdim;
  auto fetch = [&](int j0) {
    const bf16_t* kb = kx + (size_t)(j0 - x.base) * p.H * p.dim;
    const bf16_t* rb = reinterpret_cast<const bf16_t*>(p.r_cache) + (size_t)j0 * p.rot;
    const bf16_t* vb = vx + (size_t)(j0 - x.base) * p.H * p.vdim;
    const int n = last - j0;  // nothing is read past the call's last row
#pragma unroll
    for (int i = 0; i < KI; ++i) kreg[i] = *reinterpret_cast<const l_u32x4*>((krot[i] ? rb : kb) + (size_t)min(krow[i], n) * kstr[i] + kcol[i]);
#pragma unroll
    for (int i = 0; i < VI; ++i)
#pragma unroll
      for (int b = 0; b < 2; ++b) vreg[i][b] = *reinterpret_cast<const l_u32x4*>(vb + (size_t)min(vrow[i] + b, n) * p.H * p.vdim + vcol[i]);
  };
  const unsigned win = p.window > 0 ? (unsigned)p.window : 0x7fffffffu;
  // padding channels of the tiles stay zero
  for (int i = tid; i < BKV * LK / 8; i += 256) reinterpret_cast<uint4*>(&Ks[0][0])[i] = make_uint4(0, 0, 0, 0);
  if (p.vdim < VT * 16)
    for (int i = tid; i < VT * 16 * LV / 8; i += 256) reinterpret_cast<uint4*>(&Vt[0][0])[i] = make_uint4(0, 0, 0, 0);
  fetch(wb0 * BKV);
  for (int ib = 0; ib < nblocks; ++ib) {
    const int j0 = (wb0 + ib) * BKV;
    __syncthreads();
#pragma unroll
    for (int i = 0; i < KI; ++i)
      if (kin[i]) *reinterpret_cast<l_u32x4*>(&Ks[krow[i]][8 * ((tid + 256 * i) % (4 * KD))]) = kreg[i];
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
    if (ib + 1 < nblocks) fetch(j0 + BKV);
    // scores: key j0 + 16 kt + 4 lg + r of this lane's queries
    l_f32x4 sc[S][4];
#pragma unroll
    for (int kt = 0; kt < 4; ++kt) {
#pragma unroll
      for (int s = 0; s < S; ++s) sc[s][kt] = l_f32x4{0.f, 0.f, 0.f, 0.f};
      l_bf16x8 kf[KD];
#pragma unroll
      for (int kk = 0; kk < KD; ++kk) kf[kk] = *reinterpret_cast<const l_bf16x8*>(&Ks[16 * kt + l16][32 * kk + 8 * lg]);
#pragma unroll
      for (int kk = 0; kk < KD; ++kk)
#pragma unroll
        for (int s = 0; s < S; ++s) sc[s][kt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(kf[kk], qf[s][kk], sc[s][kt], 0, 0, 0);
    }
    // every row of the tile sees the whole block: inside everyone's window, before everyone
    const bool whole = j0 + BKV - 1 <= first && (p.window <= 0 || last - j0 < p.window);
    if (!whole) {
#pragma unroll
      for (int kt = 0; kt < 4; ++kt)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
          const int j = j0 + 16 * kt + 4 * lg + r;
#pragma unroll
          for (int s = 0; s < S; ++s) sc[s][kt][r] = (unsigned)(pos[s] - j) < win ? sc[s][kt][r] : -DM_INF;
        }
    }
    l_bf16x8 ph[S][2], pl[S][2];
#pragma unroll
    for (int s = 0; s < S; ++s) {
      float top = sc[s][0][0];
#pragma unroll
      for (int kt = 0; kt < 4; ++kt)
#pragma unroll
        for (int r = 0; r < 4; ++r) top = __builtin_fmaxf(top, sc[s][kt][r]);
      top = dm_max_groups16(top) * s2;
      // the reference point of a row's exponentials moves only when its maximum has grown by 2^8 (the
      // weights stay below 2^8 then, the sums far inside fp32's range)
      if (__any(top > mx[s] + 8.0f)) {
        const float mn = __builtin_fmaxf(mx[s], top), alpha = mn == -DM_INF ? 0.f : dm_exp2_hw(mx[s] - mn);
        mx[s] = mn;
        sum[s] *= alpha;
#pragma unroll
        for (int v = 0; v < VT; ++v) acc[s][v] *= alpha;
      }
      const float ref = mx[s] == -DM_INF ? 0.f : mx[s];
      float l = 0.f;
#pragma unroll
      for (int a = 0; a < 2; ++a) {
        uint32_t hi[4], lo2[4];
#pragma unroll
        for (int b = 0; b < 2; ++b) {
          float e[4];
#pragma unroll
          for (int r = 0; r < 4; ++r) {
            e[r] = dm_exp2_hw(dm_fma(sc[s][2 * a + b][r], s2, -ref));
            l += e[r];
          }
          split2(e[0], e[1], hi[2 * b], lo2[2 * b]);
          split2(e[2], e[3], hi[2 * b + 1], lo2[2 * b + 1]);
        }
        const l_u32x4 hv = {hi[0], hi[1], hi[2], hi[3]}, lv = {lo2[0], lo2[1], lo2[2], lo2[3]};
        ph[s][a] = __builtin_bit_cast(l_bf16x8, hv);
        pl[s][a] = __builtin_bit_cast(l_bf16x8, lv);
      }
      sum[s] += l;
    }
#pragma unroll
    for (int v = 0; v < VT; ++v) {
      l_bf16x8 vf[2];
#pragma unroll
      for (int a = 0; a < 2; ++a) vf[a] = *reinterpret_cast<const l_bf16x8*>(&Vt[16 * v + l16][32 * a + 8 * lg]);
#pragma unroll
      for (int a = 0; a < 2; ++a)
#pragma unroll
        for (int s = 0; s < S; ++s) acc[s][v] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf[a], ph[s][a], acc[s][v], 0, 0, 0);
#pragma unroll
      for (int a = 0; a < 2; ++a)
#pragma unroll
        for (int s = 0; s < S; ++s) acc[s][v] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(vf[a], pl[s][a], acc[s][v], 0, 0, 0);
    }
  }
#pragma unroll
  for (int s = 0; s < S; ++s) {
    const float inv = 1.0f / dm_sum_groups16(sum[s]);
    if (tq[s] >= p.T) continue;
    const float gt = inv * gate_at(p, tq[s], h);
    bf16_t* dst = reinterpret_cast<bf16_t*>(p.out) + ((size_t)tq[s] * p.H + h) * p.vdim;
#pragma unroll
    for (int v = 0; v < VT; ++v) {
      const int c = 16 * v + 4 * lg;
      if (c < p.vdim) {
        const float o[4] = {acc[s][v][0] * gt, acc[s][v][1] * gt, acc[s][v][2] * gt, acc[s][v][3] * gt};
        act_store4(dst + c, o);
      }
    }
  }
}

template <int KD, int S>
void launch_prefill(ornith_ctx* ctx, const LaArgs& p, const Expanded& x) {
  const dim3 grid(p.H, (p.T + 64 * S - 1) / (64 * S));
  if (p.vdim <= 64)
    hipLaunchKernelGGL((latent_prefill_kernel<KD, 4, S>), grid, dim3(256), 0, ctx->stream, p, x);
  else if (p.vdim <= 128)
    hipLaunchKernelGGL((latent_prefill_kernel<KD, 8, S>), grid, dim3(256), 0, ctx->stream, p, x);
  else
    hipLaunchKernelGGL((latent_prefill_kernel<KD, 16, S>), grid, dim3(256), 0, ctx->stream, p, x);
}

template <int S>
void launch_prefill_kd(ornith_ctx* ctx, const LaArgs& p, const Expanded& x, int steps) {
  if (steps <= 2) launch_prefill<2, S>(ctx, p, x);
  else if (steps <= 3) launch_prefill<3, S>(ctx, p, x);
  else if (steps <= 4) launch_prefill<4, S>(ctx, p, x);
  else if (steps <= 6) launch_prefill<6, S>(ctx, p, x);
  else launch_prefill<8, S>(ctx, p, x);
}

int run_prefill(ornith_ctx* ctx, const ornith_latent_attn_call* c, const LaArgs& p, int steps) {
  const int seen = p.window > 0 && p.offset - p.window + 1 > 0 ? p.offset - p.window + 1 : 0;
  const int base = seen / BKV * BKV, rows = p.offset + p.T - base;
  const size_t nk = (size_t)rows * p.H * p.dim, nv = (size_t)rows * p.H * p.vdim;
  void* mem = nullptr;
  int rc = ornith_scratch(ctx, (nk + nv) * 2 + 4 * 256, &mem);
  if (rc) return rc;
  ScratchCursor sc(mem);
  bf16_t* k = sc.take<bf16_t>(nk);
  bf16_t* v = sc.take<bf16_t>(nv);
  if (p.down) {
    hipLaunchKernelGGL(latent_append_kernel, dim3(p.T), dim3(NT), 0, ctx->stream, p);
    ORN_LAUNCH_CHECK("latent_append_kernel");
  }
  ornith_dense_call e{};
  e.act = ORNITH_BF16;
  e.d_x = reinterpret_cast<const bf16_t*>(p.c_cache) + (size_t)base * p.rank;
  e.M = rows;
  e.K = p.rank;
  e.n = 2;
  e.w[0] = c->uk;
  e.d_y[0] = k;
  e.w[1] = c->uv;
  e.d_y[1] = v;
  rc = ornith_dense_rows(ctx, &e);
  if (rc) return rc;
  const Expanded x{k, v, base};
  const int cus = ctx->compute_units > 0 ? ctx->compute_units : 256;
  if ((long)p.H * ((p.T + 127) / 128) >= cus) launch_prefill_kd<2>(ctx, p, x, steps);
  else launch_prefill_kd<1>(ctx, p, x, steps);
  ORN_LAUNCH_CHECK("latent_prefill_kernel");
  return ORNITH_OK;
}

}  // namespace

extern "C" int ornith_latent_attn(ornith_ctx* ctx, const ornith_latent_attn_call* c) {
  ORN_REQUIRE(ctx && c && c->d_q && c->uk && c->uv && c->d_cos && c->d_sin && c->d_c_cache && c->d_r_cache && c->d_out,
              "latent_attn: null argument");
  ORN_REQUIRE(!c->d_down || c->d_down_norm, "latent_attn: norm weight missing");
  ORN_REQUIRE(c->T >= 1 && c->H >= 1 && c->H <= 65534 && c->dim >= 1 && c->vdim >= 1 && c->rank >= 1 && c->rot_dim >= 2 && c->rot_dim % 2 == 0,
              "latent_attn: T=%d H=%d dim=%d rot_dim=%d vdim=%d rank=%d", c->T, c->H, c->dim, c->rot_dim, c->vdim, c->rank);
  ORN_REQUIRE(c->uk->mode == ORNITH_LIN_DENSE && c->uk->d_w && c->uk->O == c->H * c->dim && c->uk->K == c->rank &&
                  c->uv->mode == ORNITH_LIN_DENSE && c->uv->d_w && c->uv->O == c->H * c->vdim && c->uv->K == c->rank,
              "latent_attn: maps [%d,%d] and [%d,%d] for %d heads of %d and %d over %d", c->uk->O, c->uk->K, c->uv->O, c->uv->K, c->H,
              c->dim, c->vdim, c->rank);
  ORN_REQUIRE(c->offset >= 0 && c->offset + c->T <= c->cap && c->offset + c->T <= c->table_npos,
              "latent_attn: rows [%d, %d) in a cache of %d, tables of %d", c->offset, c->offset + c->T, c->cap, c->table_npos);
  ORN_REQUIRE(c->window >= 0, "latent_attn: window %d", c->window);
  const LaArgs p{c->d_q, c->d_down, (const bf16_t*)c->d_down_norm, (const bf16_t*)c->uk->d_w, (const bf16_t*)c->uv->d_w, c->d_gate,
                 (const bf16_t*)c->d_sink, c->d_cos, c->d_sin, c->T, c->H, c->dim, c->rot_dim, c->vdim, c->rank, c->offset, c->cap,
                 c->window, c->scale, c->eps, c->d_c_cache, c->d_r_cache, c->d_out};
  const int steps = (c->dim + 31) / 32 + (c->rot_dim + 31) / 32;
  if (c->act == ORNITH_BF16 && kPrefillRows > 0 && c->T >= kPrefillRows && c->dim % 8 == 0 && c->rot_dim % 8 == 0 && c->vdim % 8 == 0 &&
      c->rank % 8 == 0 && steps <= 8 && c->vdim <= 256)
    return run_prefill(ctx, c, p, steps);
  return c->act == ORNITH_F32 ? run_decode<float>(ctx, p) : run_decode<bf16_t>(ctx, p);
}
