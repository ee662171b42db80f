// The step of a layer-list model: embedding, per layer norm -> mixer -> sum and norm -> feed-forward
// -> sum, the closing norm. The residual stream and everything a layer adds to it are fp32; activations
// are bf16, or fp32 for a model opened in 32-bit.
//
// Launches of a layer at decode widths: an mLSTM mixer is three (projections with the norm in their
// head; the memory's step; the output projection with the heads' norm and gate in its head and the
// residual sum in its tail), an attention mixer three (four past one block of keys), a feed-forward two
// (gate and up with the norm in the head and the gated gelu in the tail; down with the residual sum).
// At prefill widths the rows a norm makes are a launch of their own and the projections are matrix-core
// GEMMs with the same tails.
#include "stack.h"

#include <algorithm>

#define TRY(e)         \
  do {                 \
    int rc__ = (e);    \
    if (rc__) return rc__; \
  } while (0)

namespace {

struct StepBufs {
  float *x, *o, *s0, *s1;                 // stream; memory output; per-head scalars
  char *rows, *q, *k, *v, *g, *q_rot, *att, *act;
};

StepBufs carve(const ornith_model* m, void* base, int R, size_t* total = nullptr) {
  size_t heads = 1, nq = 0, nk = 0, nv = 0, wide = 0, rot = 0, ff = 0;
  for (const Layer& L : m->layers) {
    if (L.mixer == MIX_MLSTM) {
      const MlstmLayer& a = L.mlstm;
      heads = std::max<size_t>(heads, a.heads);
      nq = std::max<size_t>(nq, (size_t)a.heads * a.dim);
      nk = std::max<size_t>(nk, (size_t)a.heads * a.dim);
      nv = std::max<size_t>(nv, (size_t)a.heads * a.vdim);
      wide = std::max<size_t>(wide, (size_t)a.heads * a.vdim);
    } else {
      const DiffAttnLayer& a = L.dattn;
      heads = std::max<size_t>(heads, a.heads);
      nq = std::max<size_t>(nq, (size_t)a.heads * 2 * a.dim);
      nk = std::max<size_t>(nk, (size_t)a.kv_heads * 2 * a.dim);
      nv = std::max<size_t>(nv, (size_t)a.kv_heads * a.vdim);
      wide = std::max<size_t>(wide, (size_t)a.heads * a.vdim);
      rot = std::max<size_t>(rot, (size_t)a.heads * 2 * a.dim);
    }
    if (L.ffn == FF_DENSE) ff = std::max<size_t>(ff, L.dense.ff);
  }
  const size_t W = m->cfg.hidden_size, es = ornith_dtype_size(m->act_dtype);
  ScratchCursor sc(base);
  StepBufs s;
  s.x = sc.take<float>(W * R);
  s.o = sc.take<float>(wide * R);
  s.s0 = sc.take<float>(heads * R);
  s.s1 = sc.take<float>(heads * R);
  s.rows = sc.take<char>(es * std::max(W, wide) * R);
  s.q = sc.take<char>(es * nq * R);
  s.k = sc.take<char>(es * nk * R);
  s.v = sc.take<char>(es * nv * R);
  s.g = sc.take<char>(es * wide * R);
  s.q_rot = sc.take<char>(es * rot * R);
  s.att = sc.take<char>(es * wide * R);
  s.act = sc.take<char>(es * ff * R);
  if (total) *total = sc.off;
  return s;
}

// a projection call of T rows
struct Call : ornith_dense_call {
  Call(const ornith_model* m, int T, int K_, const void* x) {
    memset(static_cast<ornith_dense_call*>(this), 0, sizeof(ornith_dense_call));
    act = m->act_dtype;
    M = T;
    K = K_;
    d_x = x;
    eps = m->cfg.rms_norm_eps;
  }
  Call& norm(const void* w, void* rows) {  // weights as their distance from one
    pre = ORNITH_PRE_NORM;
    d_norm_w = w;
    w_offset = 1.f;
    d_rows = rows;
    return *this;
  }
  Call& heads(const void* w, const void* gate, int head, void* rows) {
    pre = ORNITH_PRE_HEADS;
    d_norm_w = w;
    d_gate = gate;
    head_dim = head;
    d_rows = rows;
    return *this;
  }
  Call& to(const ornith_linear& lin, void* y, int kind = ORNITH_OUT_ACT) {
    w[n] = &lin;
    d_y[n] = y;
    out[n++] = kind;
    return *this;
  }
};

int mlstm_mixer(ornith_model* m, ornith_caches* cc, const Layer& L, LayerCache& lc, const StepBufs& s, int T, bool capture) {
  ornith_ctx* ctx = m->ctx;
  const MlstmLayer& a = L.mlstm;
  Call in = Call(m, T, m->cfg.hidden_size, s.x).norm(L.input_ln, s.rows);
  in.to(a.q, s.q).to(a.k, s.k).to(a.v, s.v).to(a.g, s.g).to(a.i, s.s0, ORNITH_OUT_F32).to(a.f, s.s1, ORNITH_OUT_F32);
  TRY(ornith_dense_rows(ctx, &in));
  ornith_mlstm_call c{};
  c.act = m->act_dtype;
  c.d_q = s.q;
  c.d_k = s.k;
  c.d_v = s.v;
  c.d_gi = s.s0;
  c.d_gf = s.s1;
  c.d_bi = a.i_b;
  c.d_bf = a.f_b;
  c.gate_cap = a.gate_cap;
  c.T = T;
  c.H = a.heads;
  c.dim = a.dim;
  c.vdim = a.vdim;
  c.d_state_in = lc.state + (size_t)cc->state_cur * (L.keeps.state / 4);
  c.d_slots = lc.state;
  c.n_slots = cc->slots;
  c.first_slot = cc->state_out(0);
  c.snapshots = capture ? 1 : 0;
  c.d_o = s.o;
  TRY(ornith_mlstm(ctx, &c));
  Call out = Call(m, T, a.heads * a.vdim, s.o).heads(a.norm, s.g, a.vdim, s.rows).to(a.o, s.x, ORNITH_OUT_ADD);
  return ornith_dense_rows(ctx, &out);
}

int diff_attn_mixer(ornith_model* m, ornith_caches* cc, const Layer& L, LayerCache& lc, const StepBufs& s, int T) {
  ornith_ctx* ctx = m->ctx;
  const DiffAttnLayer& a = L.dattn;
  Call in = Call(m, T, m->cfg.hidden_size, s.x).norm(L.input_ln, s.rows);
  in.to(a.q, s.q).to(a.k, s.k).to(a.v, s.v).to(a.g, s.s0, ORNITH_OUT_F32);
  TRY(ornith_dense_rows(ctx, &in));
  const RopeTable* rot = a.rope >= 0 ? &m->ropes[a.rope] : nullptr;
  ornith_diff_attn_call c{};
  c.act = m->act_dtype;
  c.d_q = s.q;
  c.d_k = s.k;
  c.d_v = s.v;
  c.d_gate = s.s0;
  c.d_cos = rot ? rot->d_cos : nullptr;
  c.d_sin = rot ? rot->d_sin : nullptr;
  c.rope_dims = rot ? rot->dims : 0;
  c.table_npos = m->rope_npos;
  c.T = T;
  c.H = a.heads;
  c.G = a.kv_heads;
  c.dim = a.dim;
  c.vdim = a.vdim;
  c.offset = cc->offset;
  c.cap = cc->capacity;
  c.window = a.window;
  c.keep_first = a.keep_first;
  c.scale = a.scale;
  c.lambda = a.lambda;
  c.diff = a.diff;
  c.eps = m->cfg.rms_norm_eps;
  c.d_k_cache = lc.k;
  c.d_v_cache = lc.v;
  c.d_q_rot = s.q_rot;
  c.d_out = s.att;
  TRY(ornith_diff_attn(ctx, &c));
  Call out = Call(m, T, a.heads * a.vdim, s.att).to(a.o, s.x, ORNITH_OUT_ADD);
  return ornith_dense_rows(ctx, &out);
}

int dense_ff(ornith_model* m, const Layer& L, const StepBufs& s, int T) {
  Call in = Call(m, T, m->cfg.hidden_size, s.x).norm(L.post_ln, s.rows);
  in.to(L.dense.gate, s.act).to(L.dense.up, nullptr);
  in.gelu_pair = 1;
  TRY(ornith_dense_rows(m->ctx, &in));
  Call out = Call(m, T, L.dense.ff, s.act).to(L.dense.down, s.x, ORNITH_OUT_ADD);
  return ornith_dense_rows(m->ctx, &out);
}

}  // namespace

size_t stack_step_bytes(const ornith_model* m, int rows) {
  size_t n = 0;
  carve(m, nullptr, rows, &n);
  return n + 256;
}

int stack_forward(ornith_model* m, ornith_caches* cc, const uint32_t* d_tokens, int T, bool capture, void* d_hidden) {
  const StepBufs s = carve(m, m->ws_buf, m->max_rows);
  TRY(ornith_embed_rows(m->ctx, &m->embed_tokens, d_tokens, T, m->embed_scale, s.x));
  for (size_t i = 0; i < m->layers.size(); ++i) {
    const Layer& L = m->layers[i];
    if (L.mixer == MIX_MLSTM) TRY(mlstm_mixer(m, cc, L, cc->layers[i], s, T, capture));
    else TRY(diff_attn_mixer(m, cc, L, cc->layers[i], s, T));
    if (L.ffn == FF_DENSE) TRY(dense_ff(m, L, s, T));
  }
  return ornith_norm_rows(m->ctx, s.x, m->final_norm, 1.f, T, m->cfg.hidden_size, m->cfg.rms_norm_eps, m->act_dtype, d_hidden);
}

int stack_logits(ornith_model* m, const void* d_hidden, int T, void* d_logits, int dtype) {
  const bool wide = dtype == ORNITH_F32;
  if (!wide && m->act_dtype == ORNITH_F32) {
    // a 32-bit model's sums, rounded for the samplers
    const size_t n = (size_t)T * m->cfg.vocab_size;
    void* tmp = nullptr;
    TRY(ornith_scratch(m->ctx, n * 4, &tmp));
    Call c = Call(m, T, m->cfg.hidden_size, d_hidden).to(m->lm_head, tmp, ORNITH_OUT_F32);
    TRY(ornith_dense_rows(m->ctx, &c));
    return ornith_round_bf16(m->ctx, (const float*)tmp, n, d_logits);
  }
  Call c = Call(m, T, m->cfg.hidden_size, d_hidden).to(m->lm_head, d_logits, wide ? ORNITH_OUT_F32 : ORNITH_OUT_ACT);
  return ornith_dense_rows(m->ctx, &c);
}

int stack_finish_load(ornith_model* m) {
  const size_t es = ornith_dtype_size(m->act_dtype);
  for (Layer& L : m->layers) {
    if (L.mixer == MIX_MLSTM) {
      L.keeps.state = ornith_mlstm_state_floats(L.mlstm.heads, L.mlstm.dim, L.mlstm.vdim) * 4;
    } else {
      L.keeps.kv_heads = L.dattn.kv_heads;
      L.keeps.k_row = (size_t)2 * L.dattn.dim * es;
      L.keeps.v_row = (size_t)L.dattn.vdim * es;
    }
  }
  m->max_rows = kMaxRows;
  m->ws_bytes = stack_step_bytes(m, m->max_rows);
  return ornith_alloc(m->ctx, m->ws_bytes, &m->ws_buf);
}
