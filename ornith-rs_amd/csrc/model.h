// Host-side model objects: the named-tensor store, the designs and their layers, the MTP
// head, the caches and the FR-Spec head. Mirrors WeightStore (/root/reference/src/weights.rs),
// TextModel / DecoderLayer / GatedDeltaNet / Attention
// (/root/reference/src/model/qwen3_5.rs), MtpHead (/root/reference/src/model/mtp.rs),
// KvCache / GdnCache (/root/reference/src/model/cache.rs) and FrSpec
// (/root/reference/src/frspec.rs). Everything here is host bookkeeping over device
// pointers; the arithmetic lives in the .hip files.
#pragma once

#include <map>
#include <string>
#include <vector>

#include "rt.h"

struct Tensor {
  int dtype = 0;
  std::vector<int64_t> shape;
  void* d = nullptr;
  size_t bytes = 0;
  int64_t numel() const {
    int64_t n = 1;
    for (auto s : shape) n *= s;
    return n;
  }
};

// One module's entry in config.json's `quantization` block
// (/root/reference/src/weights.rs:31-37).
struct QuantSpec {
  int group_size = 0, bits = 0, mode = ORNITH_QM_AFFINE;
};
struct QuantTable {
  bool loaded = false;
  QuantSpec def;
  std::map<std::string, QuantSpec> per_module;
  // per-module override, else the top-level default (/root/reference/src/weights.rs:96-98)
  QuantSpec lookup(const std::string& path) const {
    auto it = per_module.find(path);
    return it == per_module.end() ? def : it->second;
  }
};
int quant_table_load(const std::string& model_dir, QuantTable* qt);

namespace orn_json {
struct JVal;
}
int text_config_from(const orn_json::JVal& cfg, ornith_text_config* c, int* mtp_layers);

struct ornith_weights_files;  // the mapped shards behind a store opened from a directory
struct ornith_weights;
const Tensor* ws_fault_in(const ornith_weights* ws, const std::string& name);
void ws_release_files(ornith_weights* ws);

struct ornith_weights {
  ornith_ctx* ctx = nullptr;
  // resident tensors; a store opened from a directory copies each one in on first use
  // (WeightStore::tensor, /root/reference/src/weights.rs:101-108), hence mutable
  mutable std::map<std::string, Tensor> t;
  mutable size_t total_bytes = 0;
  // set when copying a tensor in on first use failed (allocation / upload): find() then
  // returns null for a tensor that does exist, and the caller reports this code instead of
  // "no such tensor" (the message of the failing call is already recorded)
  mutable int fault_rc = 0;
  ornith_weights_files* files = nullptr;
  QuantTable quant;
  const Tensor* find(const std::string& name) const {
    auto it = t.find(name);
    if (it != t.end()) return &it->second;
    return files ? ws_fault_in(this, name) : nullptr;
  }
};

// A lookup came back null: the reason is a failed copy-in if there was one, else a missing tensor.
#define ORN_REQUIRE_TENSOR(ws, t, ...)                               \
  do {                                                               \
    if (!(t)) {                                                      \
      if ((ws)->fault_rc) {                                          \
        const int rc__ = (ws)->fault_rc;                             \
        (ws)->fault_rc = 0;                                          \
        return rc__;                                                 \
      }                                                              \
      return ornith_fail(ORNITH_ERR_INVALID, __VA_ARGS__);           \
    }                                                                \
  } while (0)

// After lookups that may legitimately come back null (an optional tensor): a failed copy-in
// is reported as itself rather than read as "the tensor is absent".
#define ORN_RETURN_FAULT(ws)               \
  do {                                     \
    if ((ws)->fault_rc) {                  \
      const int rc__ = (ws)->fault_rc;     \
      (ws)->fault_rc = 0;                  \
      return rc__;                         \
    }                                      \
  } while (0)

// Resolves module `path` into a Linear by the tensors present (k-quant / affine8 / dense).
int ws_linear(const ornith_weights* ws, const std::string& path, ornith_linear* out);
// A routed k-quant module [E, O, K].
int ws_kmatrix(const ornith_weights* ws, const std::string& path, ornith_kmatrix* out);
// A plain tensor with an expected element count and dtype.
int ws_tensor(const ornith_weights* ws, const std::string& name, int dtype, int64_t numel,
              const void** out);
// <prefix>.<e>.<suffix> for e in 0..experts copied into one [experts, ...] tensor, kept under
// "<prefix>.*.<suffix>" (WeightStore::stacked_experts, /root/reference/src/weights.rs:237-279).
int ws_stacked(const ornith_weights* ws, const std::string& prefix, const std::string& suffix,
               int experts, int dtype, int64_t numel, const void** out);
size_t ornith_dt_size(int dt);
// A bf16 matrix [O, K] under its full name, as a dense projection.
int ws_dense(const ornith_weights* ws, const std::string& name, int O, int K, ornith_linear* out);

static const int kMaxRows = 16;  // activation rows a forward may carry unless the model is told otherwise

// ---- layers ------------------------------------------------------------------------
// A layer is a mixer (what looks across tokens) and a feed-forward, either of several kinds.
enum MixerKind { MIX_GATED_DELTA, MIX_GATED_ATTN, MIX_MLSTM, MIX_DIFF_ATTN, MIX_RETENTION, MIX_LATENT_ATTN };
enum FfKind { FF_MOE, FF_DENSE, FF_NONE };

struct GdnLayer {
  ornith_linear in_proj_qkv, in_proj_z, out_proj, in_proj_a, in_proj_b;
  const void *conv1d, *dt_bias, *a_log, *norm;
};
struct AttnLayer {
  ornith_linear q_proj, k_proj, v_proj, o_proj;
  const void *q_norm, *k_norm;
};
// mlstm.hip: matrix memory with exponential gates
struct MlstmLayer {
  int heads, dim, vdim;
  float gate_cap;
  ornith_linear q, k, v, g, o, i, f;
  const void *norm, *i_b, *f_b;
};
// diff_attn.hip: two softmax maps over the same values, rotary positions, a sliding window with
// kept first tokens, one output gate a head
struct DiffAttnLayer {
  int heads, kv_heads, dim, vdim;
  int window, keep_first;  // window 0: none
  int rope;                // which of the model's rotation tables
  float scale, diff, lambda;
  ornith_linear q, k, v, g, o;
};
// retention.hip: a matrix state a head that fades by a fixed factor, rotary positions
struct RetentionLayer {
  int heads, dim, vdim;
  int rope;
  const float* d_decay;  // f32 [heads][ORNITH_DECAY_POWERS]
  ornith_linear q, k, v, g, o;
};
// latent_attn.hip: keys and values made from one low-rank row a token, a sliding window, a sink in the
// softmax, one output gate a head
struct LatentLayer {
  int heads, dim, rot_dim, vdim, rank;
  int window;  // 0: none
  int rope;
  int kv_layer;  // the layer whose cache it reads: its own index, or an earlier one's
  float scale;
  ornith_linear q, down, uk, uv, g, o;
  const void *down_norm, *sink;
};
struct DenseFf {
  int ff;
  ornith_linear gate, up, down;
};

// What a layer keeps from token to token. The caches are laid out from this alone.
struct CacheSpec {
  int kv_heads = 0;                  // KV rows: kv_heads x capacity of
  size_t k_row = 0, v_row = 0;       //   these many bytes
  int conv_taps = 0;                 // convolution window: rows kept, and
  size_t conv_row = 0;               //   bytes a row
  size_t state = 0;                  // recurrent state: bytes a slot
};

struct StackMixer;  // stack.h
struct Layer {
  MixerKind mixer = MIX_GATED_ATTN;
  const StackMixer* ops = nullptr;  // how a layer-list model runs it
  FfKind ffn = FF_MOE;
  const void *input_ln = nullptr, *post_ln = nullptr;
  CacheSpec keeps;
  GdnLayer gdn{};
  AttnLayer attn{};
  MlstmLayer mlstm{};
  DiffAttnLayer dattn{};
  RetentionLayer ret{};
  LatentLayer latent{};
  ornith_moe_weights moe{};
  DenseFf dense{};
};

// How a rotation's frequencies are stretched: all divided by `factor`, or with YaRN's ramp between the
// pairs that turn `fast` and `slow` times over `original` positions (ornith_rope_table_yarn).
struct RopeScaling {
  double factor = 1;
  bool yarn = false;
  double original = 0, fast = 0, slow = 0;
  bool operator==(const RopeScaling& o) const {
    return factor == o.factor && yarn == o.yarn && original == o.original && fast == o.fast && slow == o.slow;
  }
};
// A rotation: cos / sin of position * base^(-2i/dims), stretched
struct RopeTable {
  int dims = 0;
  double base = 0;
  RopeScaling scaling;
  float *d_cos = nullptr, *d_sin = nullptr;  // f32 [rope_npos, dims/2]
};

// ---- designs -------------------------------------------------------------------------
// One entry of the model registry. The entry whose `architecture` is config.json's
// "architecture" loads the model; an entry without one takes the files that lack the key.
struct ModelDesign {
  const char* architecture;
  const char* name;
  bool runs_f32;  // also with activations and products in 32-bit
  int (*load)(ornith_ctx* ctx, const ornith_weights* ws, const orn_json::JVal& cfg, int act_dtype, ornith_model** out);
  size_t (*step_bytes)(const ornith_model* m, int rows);
  // T tokens through the trunk, the caches' cursors still where they were (the caller moves them)
  int (*forward)(ornith_model* m, ornith_caches* cc, const uint32_t* d_tokens, int T, bool capture, void* d_hidden);
  int (*logits)(ornith_model* m, const void* d_hidden, int T, void* d_logits, int dtype);
  // the recurrent slots are walked as a ring: a forward never writes the slot it starts from
  bool state_ring;
  ModelDesign* next;
};
struct DesignEntry {
  explicit DesignEntry(ModelDesign* d);
};

// What differs between the layer-list designs around their mixers (stack.cpp).
struct StackStyle {
  float norm_offset = 0.f;           // norm weights are stored as their distance from this
  const void* embed_norm = nullptr;  // a norm on the embedded rows
  bool side_by_side = false;         // mixer and feed-forward read the same stream, each through its norm
  float residual_mult = 1.f;         // what a layer adds is multiplied by this
  int ff_act = ORNITH_PAIR_GELU;
  float logit_cap = 0.f;             // logits become cap tanh(logits / cap); 0: as they are
};

struct ornith_model {
  ornith_ctx* ctx = nullptr;
  const ModelDesign* design = nullptr;
  int act_dtype = ORNITH_BF16;  // hidden rows, activations, KV rows
  ornith_text_config cfg{};     // every design fills hidden_size, vocab_size, num_hidden_layers, rms_norm_eps
  float embed_scale = 1.f;
  ornith_linear embed_tokens{};
  ornith_linear lm_head{};
  const void* final_norm = nullptr;
  StackStyle style;
  std::vector<Layer> layers;
  std::vector<void*> owned;  // device memory made at load
  // step buffers, sized for `max_rows` activation rows
  int max_rows = 0;
  void* ws_buf = nullptr;
  size_t ws_bytes = 0;
  // rope tables, grown on demand to the largest cache capacity seen
  std::vector<RopeTable> ropes;
  int rope_npos = 0;
  int key_dim() const { return cfg.linear_num_key_heads * cfg.linear_key_head_dim; }
  int value_dim() const { return cfg.linear_num_value_heads * cfg.linear_value_head_dim; }
  int conv_dim() const { return 2 * key_dim() + value_dim(); }
  // the table of such a rotation, made at the next model_ensure_rope
  int rope_index(int dims, double base, const RopeScaling& scaling = {});
};

struct LayerCache {
  // attention
  void *k = nullptr, *v = nullptr;  // [kv_heads, cap, row]
  // gated delta
  void* conv[2] = {nullptr, nullptr};  // bf16 [K-1+max_rows, D] each
  float* state = nullptr;              // f32 [slots][the layer's state]
};

struct ornith_caches {
  ornith_model* m = nullptr;
  int capacity = 0, max_window = 0, rows = 0;  // rows: the most a forward may carry
  int slots = 0;                               // recurrent state slots
  bool growable = true;  // a forward past the capacity grows the KV tensors (else it is refused)
  std::vector<LayerCache> layers;
  // one set of cursors serves every layer: they all advance together
  int offset = 0;     // tokens held
  int conv_cur = 0;   // which conv buffer holds the live window
  int conv_off = 0;   // first row of the live K-1 rows in it
  int state_cur = 0;  // slot holding the live recurrent state
  int state_base = 0; // slot the last forward's first snapshot went to
  int last_T = 0;     // rows of the last forward (for rewind)
  bool last_capture = false;
  // slot that receives the state after token t of the next forward
  int state_out(int t) const { return m->design->state_ring ? (state_cur + 1 + t) % slots : t; }
};

struct ornith_frspec {
  ornith_model* m = nullptr;
  int n = 0, vocab = 0;
  std::vector<uint32_t> ids;
  uint32_t* d_ids = nullptr;
  ornith_linear head{};
  void* owned[3] = {nullptr, nullptr, nullptr};
};

struct ornith_mtp_head {
  ornith_model* m = nullptr;
  const void *pre_fc_norm_embedding, *pre_fc_norm_hidden, *input_ln, *post_ln, *norm;
  ornith_linear fc;
  AttnLayer attn{};
  ornith_moe_weights moe{};
  // one-layer KV cache
  void *k = nullptr, *v = nullptr;
  int capacity = 0, offset = 0;
  bool growable = true;
  void* buf = nullptr;  // step buffers
  int max_rows = 0;
  // tokens that replace the drafts (ornith_mtp_force_drafts), indexed by output position
  uint32_t* d_forced = nullptr;
  size_t n_forced = 0;
};

// grows the model's RoPE tables to cover `npos` positions
int model_ensure_rope(ornith_model* m, int npos);
// What a loop asks before it starts: `rows` rows must fit. Growable caches always say yes (they
// grow as the rows arrive); fixed ones are checked against their capacity.
inline bool caches_fit(const ornith_caches* c, size_t rows) { return c->growable || rows <= (size_t)c->capacity; }
inline bool mtp_cache_fits(const ornith_mtp_head* h, size_t rows) { return h->growable || rows <= (size_t)h->capacity; }
