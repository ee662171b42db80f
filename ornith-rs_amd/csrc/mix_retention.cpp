// The retention mixer of layer-list models (kernels: retention.hip).
#include "stack.h"

namespace {

void needs(const Layer& L, StepNeeds& n) {
  const RetentionLayer& a = L.ret;
  n.at_least(&StepNeeds::q, (size_t)a.heads * a.dim);
  n.at_least(&StepNeeds::k, (size_t)a.heads * a.dim);
  n.at_least(&StepNeeds::v, (size_t)a.heads * a.vdim);
  n.at_least(&StepNeeds::wide, (size_t)a.heads * a.vdim);
}

void keeps(const ornith_model* m, int layer, CacheSpec& out) {
  const RetentionLayer& a = m->layers[layer].ret;
  out.state = ornith_retention_state_floats(a.heads, a.dim, a.vdim) * 4;
}

StackCall input(const StackStep& st, int layer) {
  const Layer& L = st.m->layers[layer];
  const RetentionLayer& a = L.ret;
  const StepBufs& s = st.s;
  StackCall in = mixer_input(st, L);
  in.to(a.q, s.q).to(a.k, s.k).to(a.v, s.v).to(a.g, s.g);
  return in;
}

int mix(const StackStep& st, int layer) {
  const ornith_model* m = st.m;
  const Layer& L = m->layers[layer];
  const LayerCache& lc = st.cc->layers[layer];
  const RetentionLayer& a = L.ret;
  const StepBufs& s = st.s;
  const RopeTable* rot = a.rope >= 0 ? &m->ropes[a.rope] : nullptr;
  ornith_retention_call c{};
  c.act = m->act_dtype;
  c.d_q = s.q;
  c.d_k = s.k;
  c.d_v = s.v;
  c.d_cos = rot ? rot->d_cos : nullptr;
  c.d_sin = rot ? rot->d_sin : nullptr;
  c.rope_dims = rot ? rot->dims : 0;
  c.table_npos = m->rope_npos;
  c.offset = st.cc->offset;
  c.d_decay = a.d_decay;
  c.T = st.T;
  c.H = a.heads;
  c.dim = a.dim;
  c.vdim = a.vdim;
  c.d_state_in = lc.state + (size_t)st.cc->state_cur * (L.keeps.state / 4);
  c.d_slots = lc.state;
  c.n_slots = st.cc->slots;
  c.first_slot = st.cc->state_out(0);
  c.snapshots = st.capture ? 1 : 0;
  c.d_o = s.o;
  return ornith_retention(m->ctx, &c);
}

StackCall output(const StackStep& st, int layer) {
  const RetentionLayer& a = st.m->layers[layer].ret;
  StackCall out = StackCall(st, a.heads * a.vdim, st.s.o).heads(nullptr, st.s.g, ORNITH_GATE_SILU, a.vdim);
  out.to(a.o, st.s.x, ORNITH_OUT_ADD);
  return out;
}

}  // namespace

StackMixer kRetentionMixer = {needs, keeps, input, mix, output};
