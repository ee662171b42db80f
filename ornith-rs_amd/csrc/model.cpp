// What every model design shares: the registry config.json is matched against, the caches and
// the step function (forward, rewind, logits).
//
// The caches mirror /root/reference/src/model/cache.rs and the rewind
// /root/reference/src/model/qwen3_5.rs:301-349 (TrunkCapture::rewind). A design (qwen35.cpp,
// pigodra.cpp, ranavik.cpp) brings its loader, the size of its step buffers, what each of its layers keeps
// from token to token, and its forward.
//
// Cache design (differs from the reference on purpose): every cache has a fixed
// capacity and is addressed through a few host-side cursors, so taking rows back
// after a rejected draft moves integers, never bytes:
//   KV        rows [0, offset) are live; a forward appends at `offset`.
//   conv      two buffers of K-1+rows rows; a forward reads the live K-1 rows from
//             one and writes the whole concatenated window into the other; the live
//             rows afterwards are [keep, keep+K-1) of that window.
//   state     fp32 slots. In place (gated delta, `max_window` slots): a captured forward writes
//             the state after token t into slot t; the live slot afterwards is keep-1. As a ring
//             (`max_window` + 1 slots, for kernels whose workgroups share parts of the state they
//             start from): token t goes to the slot 1 + t past the live one.
// A layer says which of these it keeps, and how many bytes, in its CacheSpec.
#include "model.h"

#include <algorithm>

#include "json.h"

#define TRY(e)         \
  do {                 \
    int rc__ = (e);    \
    if (rc__) return rc__; \
  } while (0)

namespace {
ModelDesign* g_designs = nullptr;

const ModelDesign* find_design(const orn_json::JVal& cfg) {
  const orn_json::JVal* a = cfg.get("architecture");
  for (const ModelDesign* d = g_designs; d; d = d->next) {
    if (!a && !d->architecture) return d;
    if (a && d->architecture && a->kind == orn_json::JVal::Str && a->str == d->architecture) return d;
  }
  return nullptr;
}

int load_by_config(ornith_ctx* ctx, const ornith_weights* ws, const orn_json::JVal& cfg, int act_dtype,
                   ornith_model** out) {
  ORN_REQUIRE(act_dtype == ORNITH_BF16 || act_dtype == ORNITH_F32, "model_open: activation type %d", act_dtype);
  const ModelDesign* d = find_design(cfg);
  if (!d) {
    const orn_json::JVal* a = cfg.get("architecture");
    return ornith_fail(ORNITH_ERR_UNSUPPORTED, "config.json: no model of this library is called \"%s\"",
                       a && a->kind == orn_json::JVal::Str ? a->str.c_str() : "");
  }
  if (act_dtype == ORNITH_F32 && !d->runs_f32)
    return ornith_fail(ORNITH_ERR_UNSUPPORTED, "model_open: %s runs in bf16 only", d->name);
  return d->load(ctx, ws, cfg, act_dtype, out);
}
}  // namespace

DesignEntry::DesignEntry(ModelDesign* d) {
  d->next = g_designs;
  g_designs = d;
}

int ornith_model::rope_index(int dims, double base, const RopeScaling& scaling) {
  for (size_t i = 0; i < ropes.size(); ++i)
    if (ropes[i].dims == dims && ropes[i].base == base && ropes[i].scaling == scaling) return (int)i;
  RopeTable r;
  r.dims = dims;
  r.base = base;
  r.scaling = scaling;
  ropes.push_back(r);
  return (int)ropes.size() - 1;
}

int model_ensure_rope(ornith_model* m, int npos) {
  if (npos <= m->rope_npos) return ORNITH_OK;
  ornith_ctx* ctx = m->ctx;
  m->rope_npos = 0;
  for (RopeTable& r : m->ropes) {
    ornith_free(ctx, r.d_cos);
    ornith_free(ctx, r.d_sin);
    r.d_cos = r.d_sin = nullptr;
    const size_t bytes = (size_t)npos * (r.dims / 2) * 4;
    TRY(ornith_alloc(ctx, bytes, (void**)&r.d_cos));
    TRY(ornith_alloc(ctx, bytes, (void**)&r.d_sin));
    const RopeScaling& z = r.scaling;
    if (z.yarn) TRY(ornith_rope_table_yarn(ctx, npos, r.dims, r.base, z.factor, z.original, z.fast, z.slow, r.d_cos, r.d_sin));
    else TRY(ornith_rope_table_scaled(ctx, npos, r.dims, r.base, z.factor, r.d_cos, r.d_sin));
  }
  m->rope_npos = npos;
  return ORNITH_OK;
}

extern "C" {

int ornith_model_open(ornith_ctx* ctx, const ornith_weights* ws, const char* model_dir, int act_dtype,
                      ornith_model** out) {
  ORN_REQUIRE(ctx && ws && model_dir && out, "model_open: null argument");
  orn_json::JVal cfg;
  std::string err;
  if (!orn_json::json_file(std::string(model_dir) + "/config.json", &cfg, &err))
    return ornith_fail(ORNITH_ERR_IO, "config.json: %s", err.c_str());
  return load_by_config(ctx, ws, cfg, act_dtype, out);
}

int ornith_model_load_json(ornith_ctx* ctx, const ornith_weights* ws, const char* config_json, size_t len,
                           int act_dtype, ornith_model** out) {
  ORN_REQUIRE(ctx && ws && config_json && out, "model_load_json: null argument");
  orn_json::JVal cfg;
  std::string err;
  if (!orn_json::json_parse(config_json, len, &cfg, &err)) return ornith_fail(ORNITH_ERR_INVALID, "%s", err.c_str());
  return load_by_config(ctx, ws, cfg, act_dtype, out);
}

int ornith_model_describe(const ornith_model* m, ornith_model_info* out) {
  ORN_REQUIRE(m && out, "model_describe: null argument");
  memset(out, 0, sizeof *out);
  out->hidden_size = m->cfg.hidden_size;
  out->vocab_size = m->cfg.vocab_size;
  out->num_layers = (int)m->layers.size();
  out->act_dtype = m->act_dtype;
  out->max_rows = m->max_rows;
  snprintf(out->design, sizeof out->design, "%s", m->design->name);
  return ORNITH_OK;
}

int ornith_model_set_max_rows(ornith_model* m, int rows) {
  ORN_REQUIRE(m, "model_set_max_rows: null model");
  ORN_REQUIRE(rows >= kMaxRows && rows <= 8192, "model_set_max_rows: rows=%d (%d..8192)", rows, kMaxRows);
  if (rows == m->max_rows) return ORNITH_OK;
  TRY(ornith_sync(m->ctx));
  void* buf = nullptr;
  const size_t bytes = m->design->step_bytes(m, rows);
  TRY(ornith_alloc(m->ctx, bytes, &buf));
  ornith_free(m->ctx, m->ws_buf);
  m->ws_buf = buf;
  m->ws_bytes = bytes;
  m->max_rows = rows;
  return ORNITH_OK;
}

int ornith_model_destroy(ornith_model* m) {
  if (!m) return ORNITH_OK;
  ornith_free(m->ctx, m->ws_buf);
  for (RopeTable& r : m->ropes) {
    ornith_free(m->ctx, r.d_cos);
    ornith_free(m->ctx, r.d_sin);
  }
  for (void* p : m->owned) ornith_free(m->ctx, p);
  delete m;
  return ORNITH_OK;
}

// KvCache::update_and_fetch's growth (/root/reference/src/model/cache.rs:38-79): a KV tensor
// [heads, cap, row] that must hold `need` rows moves to one of a larger capacity, a multiple of
// 256 rows as the reference's steps are and at least half as large again as before (so a long
// generation copies its cache a logarithmic number of times, not once per 256 tokens). Rows
// [0, offset) of every head are carried over; what lies past them was never committed.
static int kv_new_capacity(int capacity, int need) {
  const long grown = (long)capacity + capacity / 2;
  const long want = need > grown ? need : grown;
  return (int)((want + 255) / 256 * 256);
}

static int kv_move(ornith_ctx* ctx, void** buf, int heads, size_t row, int old_cap, int new_cap, int offset) {
  void* nb = nullptr;
  TRY(ornith_alloc(ctx, (size_t)heads * new_cap * row, &nb));
  if (offset > 0) {
    hipError_t e = hipMemcpy2DAsync(nb, (size_t)new_cap * row, *buf, (size_t)old_cap * row, (size_t)offset * row,
                                    heads, hipMemcpyDeviceToDevice, ctx->stream);
    if (e != hipSuccess) {
      ornith_free(ctx, nb);
      return ornith_fail(ORNITH_ERR_HIP, "growing a KV cache: %s", hipGetErrorString(e));
    }
  }
  const int rc = ornith_sync(ctx);  // the old tensor is freed next: everything that reads it has run
  if (rc) {
    ornith_free(ctx, nb);
    return rc;
  }
  ornith_free(ctx, *buf);
  *buf = nb;
  return ORNITH_OK;
}

int ornith_caches_reserve(ornith_caches* cc, int rows) {
  ORN_REQUIRE(cc && rows >= 0, "caches_reserve: bad argument");
  if (rows <= cc->capacity) return ORNITH_OK;
  ornith_model* m = cc->m;
  const int ncap = kv_new_capacity(cc->capacity, rows);
  TRY(model_ensure_rope(m, ncap));
  for (size_t i = 0; i < cc->layers.size(); ++i) {
    const CacheSpec& s = m->layers[i].keeps;
    if (!s.kv_heads) continue;
    TRY(kv_move(m->ctx, &cc->layers[i].k, s.kv_heads, s.k_row, cc->capacity, ncap, cc->offset));
    TRY(kv_move(m->ctx, &cc->layers[i].v, s.kv_heads, s.v_row, cc->capacity, ncap, cc->offset));
  }
  cc->capacity = ncap;
  return ORNITH_OK;
}

int ornith_caches_set_growable(ornith_caches* cc, int growable) {
  ORN_REQUIRE(cc, "caches_set_growable: null caches");
  cc->growable = growable != 0;
  return ORNITH_OK;
}

int ornith_caches_capacity(const ornith_caches* cc, int* capacity_out) {
  ORN_REQUIRE(cc && capacity_out, "caches_capacity: null argument");
  *capacity_out = cc->capacity;
  return ORNITH_OK;
}

static size_t conv_bytes(const ornith_caches* cc, const CacheSpec& s) {
  return (size_t)(s.conv_taps + cc->rows) * s.conv_row;
}

int ornith_caches_create(ornith_model* m, int capacity, int max_window, ornith_caches** out) {
  ORN_REQUIRE(m && out, "caches_create: null argument");
  ORN_REQUIRE(capacity >= 1 && max_window >= 1 && max_window <= kMaxRows,
              "caches_create: capacity=%d max_window=%d (window at most %d)", capacity, max_window,
              kMaxRows);
  ornith_caches* cc = new ornith_caches();
  cc->m = m;
  cc->capacity = capacity;
  cc->max_window = max_window;
  cc->slots = m->design->state_ring ? max_window + 1 : max_window;
  cc->rows = m->max_rows;
  cc->layers.resize(m->layers.size());
  int rc = model_ensure_rope(m, capacity);
  for (size_t i = 0; i < m->layers.size() && !rc; ++i) {
    LayerCache& lc = cc->layers[i];
    const CacheSpec& s = m->layers[i].keeps;
    if (s.kv_heads) {
      rc = ornith_alloc(m->ctx, (size_t)s.kv_heads * capacity * s.k_row, &lc.k);
      if (!rc) rc = ornith_alloc(m->ctx, (size_t)s.kv_heads * capacity * s.v_row, &lc.v);
    }
    for (int b = 0; b < 2 && s.conv_row && !rc; ++b) rc = ornith_alloc(m->ctx, conv_bytes(cc, s), &lc.conv[b]);
    if (s.state && !rc) rc = ornith_alloc(m->ctx, (size_t)cc->slots * s.state, (void**)&lc.state);
  }
  if (!rc) rc = ornith_caches_reset(cc);
  if (rc) {
    ornith_caches_destroy(cc);
    return rc;
  }
  *out = cc;
  return ORNITH_OK;
}

int ornith_caches_reset(ornith_caches* cc) {
  ORN_REQUIRE(cc, "caches_reset: null caches");
  ornith_model* m = cc->m;
  for (size_t i = 0; i < cc->layers.size(); ++i) {
    LayerCache& lc = cc->layers[i];
    const CacheSpec& s = m->layers[i].keeps;
    // conv_or_zeros / state_or_zeros (src/model/cache.rs:90-133)
    if (s.conv_row) TRY(ornith_memset(m->ctx, lc.conv[0], 0, conv_bytes(cc, s)));
    if (s.state) TRY(ornith_memset(m->ctx, lc.state, 0, s.state));
  }
  cc->offset = cc->conv_cur = cc->conv_off = cc->state_cur = cc->state_base = cc->last_T = 0;
  cc->last_capture = false;
  return ORNITH_OK;
}

int ornith_caches_destroy(ornith_caches* cc) {
  if (!cc) return ORNITH_OK;
  for (auto& lc : cc->layers) {
    ornith_free(cc->m->ctx, lc.k);
    ornith_free(cc->m->ctx, lc.v);
    ornith_free(cc->m->ctx, lc.conv[0]);
    ornith_free(cc->m->ctx, lc.conv[1]);
    ornith_free(cc->m->ctx, lc.state);
  }
  delete cc;
  return ORNITH_OK;
}

int ornith_caches_offset(const ornith_caches* cc, int* offset_out) {
  ORN_REQUIRE(cc && offset_out, "caches_offset: null argument");
  *offset_out = cc->offset;
  return ORNITH_OK;
}

int ornith_model_forward(ornith_model* m, ornith_caches* cc, const uint32_t* d_tokens, int T,
                         int capture, void* d_hidden_out) {
  ORN_REQUIRE(m && cc && d_tokens && d_hidden_out, "model_forward: null argument");
  ORN_REQUIRE(cc->m == m, "model_forward: caches belong to another model");
  ORN_REQUIRE(T >= 1 && T <= m->max_rows, "model_forward: T=%d (1..%d rows a call)", T, m->max_rows);
  ORN_REQUIRE(T <= cc->rows, "model_forward: %d rows, but these caches were created for %d rows a call", T, cc->rows);
  ORN_REQUIRE(!capture || T <= cc->max_window, "model_forward: capture of %d rows, window is %d", T,
              cc->max_window);
  ORN_REQUIRE(cc->growable || cc->offset + T <= cc->capacity, "model_forward: %d + %d rows exceed cache capacity %d",
              cc->offset, T, cc->capacity);
  TRY(ornith_caches_reserve(cc, cc->offset + T));
  TRY(m->design->forward(m, cc, d_tokens, T, capture != 0, d_hidden_out));
  // every layer advanced together
  cc->conv_cur = 1 - cc->conv_cur;
  cc->conv_off = T;
  cc->state_base = cc->state_out(0);
  cc->state_cur = cc->state_out(capture ? T - 1 : 0);
  cc->offset += T;
  cc->last_T = T;
  cc->last_capture = capture != 0;
  return ORNITH_OK;
}

int ornith_model_rewind(ornith_model* m, ornith_caches* cc, int keep) {
  ORN_REQUIRE(m && cc && cc->m == m, "model_rewind: bad argument");
  ORN_REQUIRE(cc->last_capture, "model_rewind: the last forward did not capture");
  ORN_REQUIRE(keep >= 1 && keep <= cc->last_T, "model_rewind: keep=%d of %d rows", keep, cc->last_T);
  cc->offset -= cc->last_T - keep;
  cc->conv_off = keep;
  cc->state_cur = (cc->state_base + keep - 1) % cc->slots;
  cc->last_T = keep;
  return ORNITH_OK;
}

int ornith_model_logits(ornith_model* m, const void* d_hidden, int T, void* d_logits) {
  ORN_REQUIRE(m && d_hidden && d_logits, "model_logits: null argument");
  return m->design->logits(m, d_hidden, T, d_logits, ORNITH_BF16);
}

int ornith_model_logits_f32(ornith_model* m, const void* d_hidden, int T, float* d_logits) {
  ORN_REQUIRE(m && d_hidden && d_logits, "model_logits_f32: null argument");
  return m->design->logits(m, d_hidden, T, d_logits, ORNITH_F32);
}

int ornith_mtp_cache_reserve(ornith_mtp_head* h, int rows) {
  ORN_REQUIRE(h && rows >= 0, "mtp_cache_reserve: bad argument");
  if (rows <= h->capacity) return ORNITH_OK;
  const ornith_text_config& c = h->m->cfg;
  const size_t row = (size_t)c.head_dim * 2;
  const int ncap = kv_new_capacity(h->capacity, rows);
  TRY(model_ensure_rope(h->m, ncap));
  TRY(kv_move(h->m->ctx, &h->k, c.num_key_value_heads, row, h->capacity, ncap, h->offset));
  TRY(kv_move(h->m->ctx, &h->v, c.num_key_value_heads, row, h->capacity, ncap, h->offset));
  h->capacity = ncap;
  return ORNITH_OK;
}

int ornith_mtp_cache_set_growable(ornith_mtp_head* h, int growable) {
  ORN_REQUIRE(h, "mtp_cache_set_growable: null head");
  h->growable = growable != 0;
  return ORNITH_OK;
}

}  // extern "C"
