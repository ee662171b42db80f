// The differential-attention mixer of layer-list models (kernels: diff_attn.hip).
#include "stack.h"

namespace {

void needs(const Layer& L, StepNeeds& n) {
  const DiffAttnLayer& a = L.dattn;
  n.at_least(&StepNeeds::heads, a.heads);
  n.at_least(&StepNeeds::q, (size_t)a.heads * 2 * a.dim);
  n.at_least(&StepNeeds::k, (size_t)a.kv_heads * 2 * a.dim);
  n.at_least(&StepNeeds::v, (size_t)a.kv_heads * a.vdim);
  n.at_least(&StepNeeds::wide, (size_t)a.heads * a.vdim);
  n.at_least(&StepNeeds::rot, (size_t)a.heads * 2 * a.dim);
}

void keeps(const ornith_model* m, int layer, CacheSpec& out) {
  const DiffAttnLayer& a = m->layers[layer].dattn;
  const size_t es = ornith_dtype_size(m->act_dtype);
  out.kv_heads = a.kv_heads;
  out.k_row = (size_t)2 * a.dim * es;
  out.v_row = (size_t)a.vdim * es;
}

StackCall input(const StackStep& st, int layer) {
  const Layer& L = st.m->layers[layer];
  const DiffAttnLayer& a = L.dattn;
  const StepBufs& s = st.s;
  StackCall in = mixer_input(st, L);
  in.to(a.q, s.q).to(a.k, s.k).to(a.v, s.v).to(a.g, s.s0, ORNITH_OUT_F32);
  return in;
}

int mix(const StackStep& st, int layer) {
  const ornith_model* m = st.m;
  const Layer& L = m->layers[layer];
  const LayerCache& lc = st.cc->layers[layer];
  const DiffAttnLayer& a = L.dattn;
  const StepBufs& s = st.s;
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
  c.T = st.T;
  c.H = a.heads;
  c.G = a.kv_heads;
  c.dim = a.dim;
  c.vdim = a.vdim;
  c.offset = st.cc->offset;
  c.cap = st.cc->capacity;
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
  return ornith_diff_attn(m->ctx, &c);
}

StackCall output(const StackStep& st, int layer) {
  const DiffAttnLayer& a = st.m->layers[layer].dattn;
  StackCall out = StackCall(st, a.heads * a.vdim, st.s.att).to(a.o, st.s.x, ORNITH_OUT_ADD);
  return out;
}

}  // namespace

StackMixer kDiffAttnMixer = {needs, keeps, input, mix, output};
