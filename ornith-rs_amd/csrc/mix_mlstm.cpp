// The mLSTM mixer of layer-list models (kernels: mlstm.hip).
#include "stack.h"

namespace {

void needs(const Layer& L, StepNeeds& n) {
  const MlstmLayer& a = L.mlstm;
  n.at_least(&StepNeeds::heads, a.heads);
  n.at_least(&StepNeeds::q, (size_t)a.heads * a.dim);
  n.at_least(&StepNeeds::k, (size_t)a.heads * a.dim);
  n.at_least(&StepNeeds::v, (size_t)a.heads * a.vdim);
  n.at_least(&StepNeeds::wide, (size_t)a.heads * a.vdim);
}

void keeps(const ornith_model* m, int layer, CacheSpec& out) {
  const MlstmLayer& a = m->layers[layer].mlstm;
  out.state = ornith_mlstm_state_floats(a.heads, a.dim, a.vdim) * 4;
}

StackCall input(const StackStep& st, int layer) {
  const Layer& L = st.m->layers[layer];
  const MlstmLayer& a = L.mlstm;
  const StepBufs& s = st.s;
  StackCall in = mixer_input(st, L);
  in.to(a.q, s.q).to(a.k, s.k).to(a.v, s.v).to(a.g, s.g).to(a.i, s.s0, ORNITH_OUT_F32).to(a.f, s.s1, ORNITH_OUT_F32);
  return in;
}

int mix(const StackStep& st, int layer) {
  const Layer& L = st.m->layers[layer];
  const LayerCache& lc = st.cc->layers[layer];
  const MlstmLayer& a = L.mlstm;
  const StepBufs& s = st.s;
  ornith_mlstm_call c{};
  c.act = st.m->act_dtype;
  c.d_q = s.q;
  c.d_k = s.k;
  c.d_v = s.v;
  c.d_gi = s.s0;
  c.d_gf = s.s1;
  c.d_bi = a.i_b;
  c.d_bf = a.f_b;
  c.gate_cap = a.gate_cap;
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
  return ornith_mlstm(st.m->ctx, &c);
}

StackCall output(const StackStep& st, int layer) {
  const MlstmLayer& a = st.m->layers[layer].mlstm;
  StackCall out = StackCall(st, a.heads * a.vdim, st.s.o).heads(a.norm, st.s.g, ORNITH_GATE_SIGMOID, a.vdim);
  out.to(a.o, st.s.x, ORNITH_OUT_ADD);
  return out;
}

}  // namespace

StackMixer kMlstmMixer = {needs, keeps, input, mix, output};
