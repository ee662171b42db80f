// Models that are a list of layers around a 32-bit residual stream with pre-norms: a mixer (one of the
// StackMixers below) and a dense feed-forward or none, one after the other or side by side. A design's
// loader fills an ornith_model's layers and style; these are its registry entry's step functions.
#pragma once

#include <algorithm>

#include "model.h"

// A step's buffers, one set for every layer; elements of activations unless typed.
struct StepNeeds {  // elements a row
  size_t heads = 1, q = 0, k = 0, v = 0, wide = 0, rot = 0;
  void at_least(size_t StepNeeds::*f, size_t n) { this->*f = std::max(this->*f, n); }
};
struct StepBufs {
  float *x, *o, *s0, *s1;  // stream; a mixer's 32-bit rows (wide); per-head scalars
  char *rows, *q, *k, *v, *g, *q_rot, *att, *act;
};

struct StackStep {
  ornith_model* m;
  ornith_caches* cc;
  StepBufs s;
  int T;
  bool capture;
};

// a projection call of the step's rows
struct StackCall : ornith_dense_call {
  StackCall(const StackStep& st, int K_, const void* x) {
    memset(static_cast<ornith_dense_call*>(this), 0, sizeof(ornith_dense_call));
    act = st.m->act_dtype;
    M = st.T;
    K = K_;
    d_x = x;
    eps = st.m->cfg.rms_norm_eps;
    add_scale = st.m->style.residual_mult;
    d_rows = st.s.rows;
  }
  StackCall& norm(const void* w, float offset) {
    pre = ORNITH_PRE_NORM;
    d_norm_w = w;
    w_offset = offset;
    return *this;
  }
  StackCall& heads(const void* w, const void* gate, int gate_kind, int head) {
    pre = ORNITH_PRE_HEADS;
    d_norm_w = w;
    d_gate = gate;
    gate_act = gate_kind;
    head_dim = head;
    return *this;
  }
  StackCall& to(const ornith_linear& lin, void* y, int kind = ORNITH_OUT_ACT) {
    w[n] = &lin;
    d_y[n] = y;
    out[n++] = kind;
    return *this;
  }
};
// the stream through a layer's first norm
inline StackCall mixer_input(const StackStep& st, const Layer& L) {
  return StackCall(st, st.m->cfg.hidden_size, st.s.x).norm(L.input_ln, st.m->style.norm_offset);
}

// A kind of mixer.
struct StackMixer {
  void (*needs)(const Layer& L, StepNeeds& n);
  void (*keeps)(const ornith_model* m, int layer, CacheSpec& out);
  // the projections of the normed stream
  StackCall (*input)(const StackStep& st, int layer);
  // from those to the rows the output projection reads; the stream stays as it is
  int (*mix)(const StackStep& st, int layer);
  // the output projection, added to the stream
  StackCall (*output)(const StackStep& st, int layer);
};
extern StackMixer kMlstmMixer, kDiffAttnMixer, kRetentionMixer, kLatentMixer;

size_t stack_step_bytes(const ornith_model* m, int rows);
int stack_forward(ornith_model* m, ornith_caches* cc, const uint32_t* d_tokens, int T, bool capture, void* d_hidden);
int stack_logits(ornith_model* m, const void* d_hidden, int T, void* d_logits, int dtype);
// After the layers are filled in: what each keeps, the step buffers.
int stack_finish_load(ornith_model* m);
