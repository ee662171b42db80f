// The Pigodra design: config.json and the tensor names of its artifacts.
//
// config.json: "architecture": "Pigodra", "vocab", "width", "norm": {"eps"}, "embedding": {"scale"} and
// "layers", a list of {"type", "mixer", "mlp"}:
//   "mlstm"      mixer {heads, dim, vdim, gate_cap}
//   "attention"  mixer {heads, kv_heads, dim, vdim, scale, diff, mask: {size, keep_first},
//                       rot: {base, dims, scaling: {factor}}}
//   "mlp"        null, or {"kind": "dense", "ff"}
// Tensors: embed, head, final.norm; layer i: l<i>.norm1, l<i>.norm2, l<i>.mix.*, l<i>.mlp.{gate,up,down}.
#include <cmath>

#include "stack.h"
#include "stack_config.h"

namespace {

int load_mlstm(const ornith_weights* ws, const JVal* mx, const std::string& where, const std::string& p, int W, MlstmLayer* a) {
  TRY(need_int(mx, where, "heads", 1, &a->heads));
  TRY(need_int(mx, where, "dim", 1, &a->dim));
  TRY(need_int(mx, where, "vdim", 1, &a->vdim));
  TRY(need_f32(mx, where, "gate_cap", &a->gate_cap));
  ORN_REQUIRE(a->dim <= 512, "config.json: %sdim is %d (at most 512)", where.c_str(), a->dim);
  ORN_REQUIRE(a->gate_cap > 0, "config.json: %sgate_cap is %g", where.c_str(), a->gate_cap);
  const int nk = a->heads * a->dim, nv = a->heads * a->vdim;
  TRY(ws_dense(ws, p + "q", nk, W, &a->q));
  TRY(ws_dense(ws, p + "k", nk, W, &a->k));
  TRY(ws_dense(ws, p + "v", nv, W, &a->v));
  TRY(ws_dense(ws, p + "g", nv, W, &a->g));
  TRY(ws_dense(ws, p + "o", W, nv, &a->o));
  TRY(ws_dense(ws, p + "i", a->heads, W, &a->i));
  TRY(ws_dense(ws, p + "f", a->heads, W, &a->f));
  TRY(ws_tensor(ws, p + "i.b", ORNITH_DT_BF16, a->heads, &a->i_b));
  TRY(ws_tensor(ws, p + "f.b", ORNITH_DT_BF16, a->heads, &a->f_b));
  return ws_tensor(ws, p + "norm", ORNITH_DT_BF16, nv, &a->norm);
}

// sum(a * b) of two bf16 vectors of the store
int dot_of(const ornith_weights* ws, const std::string& a, const std::string& b, int n, double* out) {
  *out = 0;
  const void* d[2];
  TRY(ws_tensor(ws, a, ORNITH_DT_BF16, n, &d[0]));
  TRY(ws_tensor(ws, b, ORNITH_DT_BF16, n, &d[1]));
  std::vector<uint16_t> v[2] = {std::vector<uint16_t>(n), std::vector<uint16_t>(n)};
  for (int i = 0; i < 2; ++i) TRY(ornith_download(ws->ctx, v[i].data(), d[i], (size_t)n * 2));
  auto value = [](uint16_t bits) {
    const uint32_t u = (uint32_t)bits << 16;
    float f;
    memcpy(&f, &u, 4);
    return (double)f;
  };
  for (int i = 0; i < n; ++i) *out += value(v[0][i]) * value(v[1][i]);
  return ORNITH_OK;
}

int load_attention(ornith_model* m, const ornith_weights* ws, const JVal* mx, const std::string& where, const std::string& p,
                   int W, DiffAttnLayer* a) {
  TRY(need_int(mx, where, "heads", 1, &a->heads));
  TRY(need_int(mx, where, "kv_heads", 1, &a->kv_heads));
  TRY(need_int(mx, where, "dim", 1, &a->dim));
  TRY(need_int(mx, where, "vdim", 1, &a->vdim));
  TRY(need_f32(mx, where, "scale", &a->scale));
  TRY(need_f32(mx, where, "diff", &a->diff));
  ORN_REQUIRE(a->heads % a->kv_heads == 0, "config.json: %s%d heads over %d kv_heads", where.c_str(), a->heads, a->kv_heads);
  a->window = a->keep_first = 0;
  const JVal* mask = mx->get("mask");
  if (!absent(mask)) {
    TRY(need_int(mask, where + "mask.", "size", 1, &a->window));
    TRY(need_int(mask, where + "mask.", "keep_first", 0, &a->keep_first));
  }
  a->rope = -1;
  const JVal* rot = mx->get("rot");
  if (!absent(rot)) {
    int dims = 0;
    double base = 0, factor = 1;
    TRY(need_int(rot, where + "rot.", "dims", 0, &dims));
    TRY(need_num(rot, where + "rot.", "base", &base));
    const JVal* scaling = rot->get("scaling");
    if (!absent(scaling)) TRY(need_num(scaling, where + "rot.scaling.", "factor", &factor));
    ORN_REQUIRE(dims % 2 == 0 && dims <= a->dim && base > 0 && factor > 0, "config.json: %srot turns %d of %d dimensions, base %g, factor %g",
                where.c_str(), dims, a->dim, base, factor);
    if (dims > 0) a->rope = m->rope_index(dims, base, RopeScaling{factor});
  }
  TRY(ws_dense(ws, p + "q", a->heads * 2 * a->dim, W, &a->q));
  TRY(ws_dense(ws, p + "k", a->kv_heads * 2 * a->dim, W, &a->k));
  TRY(ws_dense(ws, p + "v", a->kv_heads * a->vdim, W, &a->v));
  TRY(ws_dense(ws, p + "g", a->heads, W, &a->g));
  TRY(ws_dense(ws, p + "o", W, a->heads * a->vdim, &a->o));
  double d1 = 0, d2 = 0;
  TRY(dot_of(ws, p + "lq1", p + "lk1", a->dim, &d1));
  TRY(dot_of(ws, p + "lq2", p + "lk2", a->dim, &d2));
  a->lambda = (float)(std::exp(d1) - std::exp(d2) + (double)a->diff);
  return ORNITH_OK;
}

int load_into(ornith_model* m, const ornith_weights* ws, const JVal& cfg) {
  ornith_text_config& c = m->cfg;
  TRY(need_int(&cfg, "", "width", 1, &c.hidden_size));
  TRY(need_int(&cfg, "", "vocab", 1, &c.vocab_size));
  TRY(need_f32(cfg.get("norm"), "norm.", "eps", &c.rms_norm_eps));
  TRY(need_f32(cfg.get("embedding"), "embedding.", "scale", &m->embed_scale));
  const int W = c.hidden_size;
  const JVal* layers = cfg.get("layers");
  ORN_REQUIRE(layers && layers->kind == JVal::Arr && !layers->arr.empty(), "config.json: no layers");
  c.num_hidden_layers = (int)layers->arr.size();
  m->layers.resize(layers->arr.size());
  TRY(ws_dense(ws, "embed", c.vocab_size, W, &m->embed_tokens));
  TRY(ws_dense(ws, "head", c.vocab_size, W, &m->lm_head));
  TRY(ws_tensor(ws, "final.norm", ORNITH_DT_BF16, W, &m->final_norm));
  for (size_t i = 0; i < layers->arr.size(); ++i) {
    const JVal& e = layers->arr[i];
    Layer& L = m->layers[i];
    const std::string p = "l" + std::to_string(i) + ".", where = "layers[" + std::to_string(i) + "].mixer.";
    const JVal *type = e.get("type"), *mx = e.get("mixer"), *mlp = e.get("mlp");
    ORN_REQUIRE(type && type->kind == JVal::Str && mx && mx->kind == JVal::Obj, "config.json: layers[%zu] needs a type and a mixer", i);
    TRY(ws_tensor(ws, p + "norm1", ORNITH_DT_BF16, W, &L.input_ln));
    if (type->str == "mlstm") {
      L.mixer = MIX_MLSTM;
      L.ops = &kMlstmMixer;
      TRY(load_mlstm(ws, mx, where, p + "mix.", W, &L.mlstm));
    } else if (type->str == "attention") {
      L.mixer = MIX_DIFF_ATTN;
      L.ops = &kDiffAttnMixer;
      TRY(load_attention(m, ws, mx, where, p + "mix.", W, &L.dattn));
    } else {
      return ornith_fail(ORNITH_ERR_UNSUPPORTED, "config.json: layers[%zu] is of type \"%s\"", i, type->str.c_str());
    }
    TRY(stack_load_ff(ws, mlp, i, W, &L));
  }
  m->style.norm_offset = 1.f;
  return stack_finish_load(m);
}

int load(ornith_ctx* ctx, const ornith_weights* ws, const JVal& cfg, int act_dtype, ornith_model** out);

ModelDesign kPigodra = {"Pigodra", "pigodra", true, load, stack_step_bytes, stack_forward, stack_logits, true, nullptr};
const DesignEntry kPigodraEntry(&kPigodra);

int load(ornith_ctx* ctx, const ornith_weights* ws, const JVal& cfg, int act_dtype, ornith_model** out) {
  ornith_model* m = new ornith_model();
  m->ctx = ctx;
  m->design = &kPigodra;
  m->act_dtype = act_dtype;
  const int rc = load_into(m, ws, cfg);
  if (rc) {
    ornith_model_destroy(m);
    return rc;
  }
  *out = m;
  return ORNITH_OK;
}

}  // namespace
