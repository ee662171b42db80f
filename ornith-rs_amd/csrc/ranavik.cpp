// The Ranavik design: config.json and the tensor names of its artifacts. Mixer and feed-forward of a layer
// stand side by side: x += residual_mult (mixer(norm1 x) + ff(norm2 x)).
//
// config.json: "architecture": "Ranavik", "vocab", "width", "norm": {"eps"}, "residual_mult",
// "logit_softcap" and "layers", a list of {"type", "mixer", "mlp"}:
//   "retention"         mixer {heads, dim, vdim, decay: [a number a head], rot: {base, dims}}
//   "latent_attention"  mixer {heads, dim, rot_dim, vdim, kv_rank, scale, mask: {size}, kv_from: an earlier
//                              layer whose cached rows this one reads, rot: {base, dims: rot_dim,
//                              scaling: {factor, original, fast, slow}}}
//   "mlp"               null, or {"kind": "dense", "ff"}
// Tensors: embed, embed.norm, head, final.norm; layer i: l<i>.norm1, l<i>.norm2, l<i>.mix.*,
// l<i>.mlp.{gate,up,down}.
#include "stack.h"
#include "stack_config.h"

namespace {

// the table of a layer's rotation (-1: nothing turns)
int load_rot(ornith_model* m, const JVal* mx, const std::string& where, int most, int* dims_out, int* rope) {
  *rope = -1;
  *dims_out = 0;
  const JVal* rot = mx->get("rot");
  if (absent(rot)) return ORNITH_OK;
  int dims = 0;
  double base = 0;
  RopeScaling z;
  TRY(need_int(rot, where + "rot.", "dims", 0, &dims));
  TRY(need_num(rot, where + "rot.", "base", &base));
  ORN_REQUIRE(dims % 2 == 0 && dims <= most && base > 0, "config.json: %srot turns %d of %d dimensions, base %g", where.c_str(), dims,
              most, base);
  const JVal* scaling = rot->get("scaling");
  if (!absent(scaling)) {
    const std::string at = where + "rot.scaling.";
    z.yarn = true;
    TRY(need_num(scaling, at, "factor", &z.factor));
    TRY(need_num(scaling, at, "original", &z.original));
    TRY(need_num(scaling, at, "fast", &z.fast));
    TRY(need_num(scaling, at, "slow", &z.slow));
    ORN_REQUIRE(z.factor > 0 && z.original > 0 && z.fast > 0 && z.slow > 0 && base != 1.0,
                "config.json: %sfactor %g, original %g, fast %g, slow %g", at.c_str(), z.factor, z.original, z.fast, z.slow);
  }
  *dims_out = dims;
  if (dims > 0) *rope = m->rope_index(dims, base, z);
  return ORNITH_OK;
}

int load_retention(ornith_model* m, const ornith_weights* ws, const JVal* mx, const std::string& where, const std::string& p,
                   int W, RetentionLayer* a) {
  TRY(need_int(mx, where, "heads", 1, &a->heads));
  TRY(need_int(mx, where, "dim", 1, &a->dim));
  TRY(need_int(mx, where, "vdim", 1, &a->vdim));
  ORN_REQUIRE(a->dim <= 512, "config.json: %sdim is %d (at most 512)", where.c_str(), a->dim);
  int turned = 0;
  TRY(load_rot(m, mx, where, a->dim, &turned, &a->rope));
  const JVal* decay = mx->get("decay");
  ORN_REQUIRE(decay && decay->kind == JVal::Arr && decay->arr.size() == (size_t)a->heads,
              "config.json: %sdecay must list a number for each of %d heads", where.c_str(), a->heads);
  std::vector<double> d;
  for (const JVal& v : decay->arr) {
    ORN_REQUIRE(v.kind == JVal::Num, "config.json: %sdecay holds something that is no number", where.c_str());
    d.push_back(v.num);
  }
  void* table = nullptr;
  TRY(ornith_alloc(m->ctx, (size_t)a->heads * ORNITH_DECAY_POWERS * 4, &table));
  m->owned.push_back(table);
  TRY(ornith_decay_powers(m->ctx, a->heads, d.data(), (float*)table));
  a->d_decay = (const float*)table;
  const int nk = a->heads * a->dim, nv = a->heads * a->vdim;
  TRY(ws_dense(ws, p + "q", nk, W, &a->q));
  TRY(ws_dense(ws, p + "k", nk, W, &a->k));
  TRY(ws_dense(ws, p + "v", nv, W, &a->v));
  TRY(ws_dense(ws, p + "g", nv, W, &a->g));
  return ws_dense(ws, p + "o", W, nv, &a->o);
}

int load_latent(ornith_model* m, const ornith_weights* ws, const JVal* mx, const std::string& where, const std::string& p, int W,
                int layer, LatentLayer* a) {
  TRY(need_int(mx, where, "heads", 1, &a->heads));
  TRY(need_int(mx, where, "dim", 1, &a->dim));
  TRY(need_int(mx, where, "rot_dim", 1, &a->rot_dim));
  TRY(need_int(mx, where, "vdim", 1, &a->vdim));
  TRY(need_int(mx, where, "kv_rank", 1, &a->rank));
  TRY(need_f32(mx, where, "scale", &a->scale));
  a->window = 0;
  const JVal* mask = mx->get("mask");
  if (!absent(mask)) TRY(need_int(mask, where + "mask.", "size", 1, &a->window));
  int turned = 0;
  TRY(load_rot(m, mx, where, a->rot_dim, &turned, &a->rope));
  ORN_REQUIRE(turned == a->rot_dim, "config.json: %srot turns %d of %d rotated dimensions", where.c_str(), turned, a->rot_dim);
  a->kv_layer = layer;
  if (!absent(mx->get("kv_from"))) {
    TRY(need_int(mx, where, "kv_from", 0, &a->kv_layer));
    const Layer* from = a->kv_layer < layer ? &m->layers[a->kv_layer] : nullptr;
    ORN_REQUIRE(from && from->mixer == MIX_LATENT_ATTN && from->latent.kv_layer == a->kv_layer,
                "config.json: %skv_from is %d, no earlier latent_attention layer with a cache of its own", where.c_str(), a->kv_layer);
    ORN_REQUIRE(from->latent.rank == a->rank && from->latent.rot_dim == a->rot_dim && from->latent.rope == a->rope,
                "config.json: %skv_rank, rot_dim or rot differ from those of layer %d", where.c_str(), a->kv_layer);
  }
  const int H = a->heads;
  TRY(ws_dense(ws, p + "q", H * (a->dim + a->rot_dim), W, &a->q));
  if (a->kv_layer == layer) {
    TRY(ws_dense(ws, p + "dkv", a->rank + a->rot_dim, W, &a->down));
    TRY(ws_tensor(ws, p + "dkv.norm", ORNITH_DT_BF16, a->rank, &a->down_norm));
  }
  TRY(ws_dense(ws, p + "uk", H * a->dim, a->rank, &a->uk));
  TRY(ws_dense(ws, p + "uv", H * a->vdim, a->rank, &a->uv));
  TRY(ws_tensor(ws, p + "sink", ORNITH_DT_BF16, H, &a->sink));
  TRY(ws_dense(ws, p + "g", H, W, &a->g));
  return ws_dense(ws, p + "o", W, H * a->vdim, &a->o);
}

int load_into(ornith_model* m, const ornith_weights* ws, const JVal& cfg) {
  ornith_text_config& c = m->cfg;
  StackStyle& y = m->style;
  TRY(need_int(&cfg, "", "width", 1, &c.hidden_size));
  TRY(need_int(&cfg, "", "vocab", 1, &c.vocab_size));
  TRY(need_f32(cfg.get("norm"), "norm.", "eps", &c.rms_norm_eps));
  TRY(need_f32(&cfg, "", "residual_mult", &y.residual_mult));
  if (!absent(cfg.get("logit_softcap"))) {
    TRY(need_f32(&cfg, "", "logit_softcap", &y.logit_cap));
    ORN_REQUIRE(y.logit_cap > 0, "config.json: logit_softcap is %g", y.logit_cap);
  }
  y.side_by_side = true;
  y.ff_act = ORNITH_PAIR_SILU;
  const int W = c.hidden_size;
  const JVal* layers = cfg.get("layers");
  ORN_REQUIRE(layers && layers->kind == JVal::Arr && !layers->arr.empty(), "config.json: no layers");
  c.num_hidden_layers = (int)layers->arr.size();
  m->layers.resize(layers->arr.size());
  TRY(ws_dense(ws, "embed", c.vocab_size, W, &m->embed_tokens));
  TRY(ws_tensor(ws, "embed.norm", ORNITH_DT_BF16, W, &y.embed_norm));
  TRY(ws_dense(ws, "head", c.vocab_size, W, &m->lm_head));
  TRY(ws_tensor(ws, "final.norm", ORNITH_DT_BF16, W, &m->final_norm));
  for (size_t i = 0; i < layers->arr.size(); ++i) {
    const JVal& e = layers->arr[i];
    Layer& L = m->layers[i];
    const std::string p = "l" + std::to_string(i) + ".", where = "layers[" + std::to_string(i) + "].mixer.";
    const JVal *type = e.get("type"), *mx = e.get("mixer");
    ORN_REQUIRE(type && type->kind == JVal::Str && mx && mx->kind == JVal::Obj, "config.json: layers[%zu] needs a type and a mixer", i);
    TRY(ws_tensor(ws, p + "norm1", ORNITH_DT_BF16, W, &L.input_ln));
    if (type->str == "retention") {
      L.mixer = MIX_RETENTION;
      L.ops = &kRetentionMixer;
      TRY(load_retention(m, ws, mx, where, p + "mix.", W, &L.ret));
    } else if (type->str == "latent_attention") {
      L.mixer = MIX_LATENT_ATTN;
      L.ops = &kLatentMixer;
      TRY(load_latent(m, ws, mx, where, p + "mix.", W, (int)i, &L.latent));
    } else {
      return ornith_fail(ORNITH_ERR_UNSUPPORTED, "config.json: layers[%zu] is of type \"%s\"", i, type->str.c_str());
    }
    TRY(stack_load_ff(ws, e.get("mlp"), i, W, &L));
  }
  return stack_finish_load(m);
}

int load(ornith_ctx* ctx, const ornith_weights* ws, const JVal& cfg, int act_dtype, ornith_model** out);

ModelDesign kRanavik = {"Ranavik", "ranavik", true, load, stack_step_bytes, stack_forward, stack_logits, true, nullptr};
const DesignEntry kRanavikEntry(&kRanavik);

int load(ornith_ctx* ctx, const ornith_weights* ws, const JVal& cfg, int act_dtype, ornith_model** out) {
  ornith_model* m = new ornith_model();
  m->ctx = ctx;
  m->design = &kRanavik;
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
