// The step of a layer-list model: embedding (and its norm), the layers, the closing norm. The residual
// stream and everything a layer adds to it are fp32; activations are bf16, or fp32 for a model opened in
// 32-bit. A layer is norm -> mixer -> sum, norm -> feed-forward -> sum, or both halves side by side on the
// same stream: then the projections behind both norms come first, in one launch at decode widths.
//
// Launches of a layer at decode widths: a recurrent mixer is three (projections with the norm in their
// head; the memory's step; the output projection with the heads' norm and gate in its head and the
// residual sum in its tail), differential attention three (four past one block of keys), latent attention
// five, a feed-forward two (gate and up with the norm in the head and the activation in the tail; down with
// the residual sum), of which only the second is a launch of its own beside a mixer. At prefill widths the
// rows a norm makes are a launch of their own and the projections are matrix-core GEMMs with the same tails.
#include "stack.h"

#define TRY(e)         \
  do {                 \
    int rc__ = (e);    \
    if (rc__) return rc__; \
  } while (0)

namespace {

StepBufs carve(const ornith_model* m, void* base, int R, size_t* total = nullptr) {
  StepNeeds n;
  size_t ff = 0;
  for (const Layer& L : m->layers) {
    L.ops->needs(L, n);
    if (L.ffn == FF_DENSE) ff = std::max<size_t>(ff, L.dense.ff);
  }
  const size_t W = m->cfg.hidden_size, es = ornith_dtype_size(m->act_dtype);
  ScratchCursor sc(base);
  StepBufs s;
  s.x = sc.take<float>(W * R);
  s.o = sc.take<float>(n.wide * R);
  s.s0 = sc.take<float>(n.heads * R);
  s.s1 = sc.take<float>(n.heads * R);
  s.rows = sc.take<char>(es * std::max(W, n.wide) * R);
  s.q = sc.take<char>(es * n.q * R);
  s.k = sc.take<char>(es * n.k * R);
  s.v = sc.take<char>(es * n.v * R);
  s.g = sc.take<char>(es * n.wide * R);
  s.q_rot = sc.take<char>(es * n.rot * R);
  s.att = sc.take<char>(es * n.wide * R);
  s.act = sc.take<char>(es * ff * R);
  if (total) *total = sc.off;
  return s;
}

int run(const StackStep& st, const StackCall& c) { return ornith_dense_rows(st.m->ctx, &c); }

StackCall ff_in(const StackStep& st, const Layer& L) {
  StackCall c = StackCall(st, st.m->cfg.hidden_size, st.s.x).norm(L.post_ln, st.m->style.norm_offset);
  c.to(L.dense.gate, st.s.act).to(L.dense.up, nullptr);
  c.pair_act = st.m->style.ff_act;
  return c;
}

StackCall ff_out(const StackStep& st, const Layer& L) {
  return StackCall(st, L.dense.ff, st.s.act).to(L.dense.down, st.s.x, ORNITH_OUT_ADD);
}

}  // namespace

size_t stack_step_bytes(const ornith_model* m, int rows) {
  size_t n = 0;
  carve(m, nullptr, rows, &n);
  return n + 256;
}

int stack_forward(ornith_model* m, ornith_caches* cc, const uint32_t* d_tokens, int T, bool capture, void* d_hidden) {
  const StackStep st{m, cc, carve(m, m->ws_buf, m->max_rows), T, capture};
  const StackStyle& y = m->style;
  if (y.embed_norm)
    TRY(ornith_embed_norm_rows(m->ctx, &m->embed_tokens, d_tokens, T, y.embed_norm, y.norm_offset, m->cfg.rms_norm_eps, st.s.x));
  else
    TRY(ornith_embed_rows(m->ctx, &m->embed_tokens, d_tokens, T, m->embed_scale, st.s.x));
  for (int i = 0; i < (int)m->layers.size(); ++i) {
    const Layer& L = m->layers[i];
    const bool ff = L.ffn == FF_DENSE;
    const StackCall in = L.ops->input(st, i);
    if (ff && y.side_by_side) {
      const StackCall up = ff_in(st, L);
      TRY(ornith_dense_rows_duo(m->ctx, &in, &up));
    } else {
      TRY(run(st, in));
    }
    TRY(L.ops->mix(st, i));
    TRY(run(st, L.ops->output(st, i)));
    if (ff && !y.side_by_side) TRY(run(st, ff_in(st, L)));
    if (ff) TRY(run(st, ff_out(st, L)));
  }
  return ornith_norm_rows(m->ctx, st.s.x, m->final_norm, y.norm_offset, T, m->cfg.hidden_size, m->cfg.rms_norm_eps,
                          m->act_dtype, d_hidden);
}

int stack_logits(ornith_model* m, const void* d_hidden, int T, void* d_logits, int dtype) {
  const bool wide = dtype == ORNITH_F32;
  const StackStep st{m, nullptr, {}, T, false};
  StackCall c(st, m->cfg.hidden_size, d_hidden);
  c.soft_cap = m->style.logit_cap;
  if (!wide && m->act_dtype == ORNITH_F32) {
    // a 32-bit model's sums, rounded for the samplers
    const size_t n = (size_t)T * m->cfg.vocab_size;
    void* tmp = nullptr;
    TRY(ornith_scratch(m->ctx, n * 4, &tmp));
    c.to(m->lm_head, tmp, ORNITH_OUT_F32);
    TRY(ornith_dense_rows(m->ctx, &c));
    return ornith_round_bf16(m->ctx, (const float*)tmp, n, d_logits);
  }
  c.to(m->lm_head, d_logits, wide ? ORNITH_OUT_F32 : ORNITH_OUT_ACT);
  return ornith_dense_rows(m->ctx, &c);
}

int stack_finish_load(ornith_model* m) {
  for (int i = 0; i < (int)m->layers.size(); ++i) m->layers[i].ops->keeps(m, i, m->layers[i].keeps);
  m->max_rows = kMaxRows;
  m->ws_bytes = stack_step_bytes(m, m->max_rows);
  return ornith_alloc(m->ctx, m->ws_bytes, &m->ws_buf);
}
