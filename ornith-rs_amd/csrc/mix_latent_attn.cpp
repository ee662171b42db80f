// The latent-attention mixer of layer-list models (kernels: latent_attn.hip). A layer that reads an earlier
// layer's cache has no down projection and keeps nothing itself.
#include "stack.h"

namespace {

void needs(const Layer& L, StepNeeds& n) {
  const LatentLayer& a = L.latent;
  n.at_least(&StepNeeds::heads, a.heads);
  n.at_least(&StepNeeds::q, (size_t)a.heads * (a.dim + a.rot_dim));
  n.at_least(&StepNeeds::wide, std::max((size_t)a.heads * a.vdim, (size_t)a.rank + a.rot_dim));
}

void keeps(const ornith_model* m, int layer, CacheSpec& out) {
  const LatentLayer& a = m->layers[layer].latent;
  if (a.kv_layer != layer) return;
  const size_t es = ornith_dtype_size(m->act_dtype);
  out.kv_heads = 1;
  out.k_row = (size_t)a.rank * es;
  out.v_row = (size_t)a.rot_dim * es;
}

StackCall input(const StackStep& st, int layer) {
  const Layer& L = st.m->layers[layer];
  const LatentLayer& a = L.latent;
  const StepBufs& s = st.s;
  StackCall in = mixer_input(st, L);
  in.to(a.q, s.q).to(a.g, s.s0, ORNITH_OUT_F32);
  if (a.kv_layer == layer) in.to(a.down, s.o, ORNITH_OUT_F32);
  return in;
}

int mix(const StackStep& st, int layer) {
  const ornith_model* m = st.m;
  const Layer& L = m->layers[layer];
  const LatentLayer& a = L.latent;
  const LayerCache& lc = st.cc->layers[a.kv_layer];
  const StepBufs& s = st.s;
  const bool own = a.kv_layer == layer;
  const RopeTable* rot = a.rope >= 0 ? &m->ropes[a.rope] : nullptr;
  ornith_latent_attn_call c{};
  c.act = m->act_dtype;
  c.d_q = s.q;
  c.d_down = own ? s.o : nullptr;
  c.d_down_norm = a.down_norm;
  c.uk = &a.uk;
  c.uv = &a.uv;
  c.d_gate = s.s0;
  c.d_sink = a.sink;
  c.d_cos = rot ? rot->d_cos : nullptr;
  c.d_sin = rot ? rot->d_sin : nullptr;
  c.table_npos = m->rope_npos;
  c.T = st.T;
  c.H = a.heads;
  c.dim = a.dim;
  c.rot_dim = a.rot_dim;
  c.vdim = a.vdim;
  c.rank = a.rank;
  c.offset = st.cc->offset;
  c.cap = st.cc->capacity;
  c.window = a.window;
  c.scale = a.scale;
  c.eps = m->cfg.rms_norm_eps;
  c.d_c_cache = lc.k;
  c.d_r_cache = lc.v;
  c.d_out = s.att;
  return ornith_latent_attn(m->ctx, &c);
}

StackCall output(const StackStep& st, int layer) {
  const LatentLayer& a = st.m->layers[layer].latent;
  StackCall out = StackCall(st, a.heads * a.vdim, st.s.att).to(a.o, st.s.x, ORNITH_OUT_ADD);
  return out;
}

}  // namespace

StackMixer kLatentMixer = {needs, keeps, input, mix, output};
