// What the loaders of the layer-list designs read config.json with.
#pragma once

#include <climits>

#include "json.h"
#include "model.h"

#define TRY(e)         \
  do {                 \
    int rc__ = (e);    \
    if (rc__) return rc__; \
  } while (0)

using orn_json::JVal;

inline int need_num(const JVal* o, const std::string& where, const char* key, double* out) {
  const JVal* j = o ? o->get(key) : nullptr;
  ORN_REQUIRE(j && j->kind == JVal::Num, "config.json: missing %s%s", where.c_str(), key);
  *out = j->num;
  return ORNITH_OK;
}

inline int need_f32(const JVal* o, const std::string& where, const char* key, float* out) {
  double v = 0;
  TRY(need_num(o, where, key, &v));
  *out = (float)v;
  return ORNITH_OK;
}

inline int need_int(const JVal* o, const std::string& where, const char* key, int min, int* out) {
  const JVal* j = o ? o->get(key) : nullptr;
  size_t v = 0;
  ORN_REQUIRE(j && j->as_usize(&v), "config.json: missing %s%s", where.c_str(), key);
  ORN_REQUIRE(v >= (size_t)min && v <= INT_MAX / 2, "config.json: %s%s is %zu", where.c_str(), key, v);
  *out = (int)v;
  return ORNITH_OK;
}

inline bool absent(const JVal* j) { return !j || j->kind == JVal::Null; }

// A layer's dense feed-forward, or none: its norm l<i>.norm2 and l<i>.mlp.{gate, up, down}.
inline int stack_load_ff(const ornith_weights* ws, const JVal* mlp, size_t i, int W, Layer* L) {
  L->ffn = FF_NONE;
  if (absent(mlp)) return ORNITH_OK;
  const std::string p = "l" + std::to_string(i) + ".";
  const JVal* kind = mlp->get("kind");
  if (!(kind && kind->kind == JVal::Str && kind->str == "dense"))
    return ornith_fail(ORNITH_ERR_UNSUPPORTED, "config.json: layers[%zu].mlp is of a kind this design does not have", i);
  L->ffn = FF_DENSE;
  TRY(need_int(mlp, "layers[" + std::to_string(i) + "].mlp.", "ff", 1, &L->dense.ff));
  TRY(ws_tensor(ws, p + "norm2", ORNITH_DT_BF16, W, &L->post_ln));
  TRY(ws_dense(ws, p + "mlp.gate", L->dense.ff, W, &L->dense.gate));
  TRY(ws_dense(ws, p + "mlp.up", L->dense.ff, W, &L->dense.up));
  return ws_dense(ws, p + "mlp.down", W, L->dense.ff, &L->dense.down);
}
