// Shared by the generation loops (engine.cpp, mtp_engine.cpp): a call's device buffers, the
// sampler a loop drives, and the prompt's prefill.
#pragma once

#include <algorithm>
#include <vector>

#include "model.h"

#define LOOP_TRY(e)        \
  do {                     \
    int rc__ = (e);        \
    if (rc__) return rc__; \
  } while (0)

// device buffers a generation call needs, freed on scope exit
struct Bufs {
  ornith_ctx* ctx;
  std::vector<void*> all;
  explicit Bufs(ornith_ctx* c) : ctx(c) {}
  ~Bufs() {
    for (void* p : all) ornith_free(ctx, p);
  }
  int get(size_t bytes, void** out) {
    int rc = ornith_alloc(ctx, bytes, out);
    if (!rc) all.push_back(*out);
    return rc;
  }
};

// The `Sampler` a loop drives (src/generate.rs:36-64): Greedy, or TopSampler built from
// the tagged struct. rows_are_independent() is true for Greedy only: every draw of the
// other advances its key, so rows are sampled one by one and only when asked for.
struct LoopSampler {
  ornith_ctx* ctx = nullptr;
  ornith_top_sampler* top = nullptr;
  int V = 0;
  bool ratio = false;  // drafts drawn from the head's distribution and accepted by probability ratio
  ~LoopSampler() {
    if (top) ornith_top_sampler_destroy(top);
  }
  int init(ornith_ctx* c, const ornith_sampler* s, int vocab) {
    ORN_REQUIRE(s, "sampler is null");
    ctx = c;
    V = vocab;
    if (s->kind == ORNITH_SAMPLER_GREEDY) return ORNITH_OK;
    ORN_REQUIRE(s->kind == ORNITH_SAMPLER_TOP_P, "unknown sampler kind %d", s->kind);
    ORN_REQUIRE(s->accept == ORNITH_ACCEPT_EQUALITY || s->accept == ORNITH_ACCEPT_RATIO,
                "unknown acceptance rule %d", s->accept);
    ORN_REQUIRE(s->rng == ORNITH_RNG_THREEFRY || s->rng == ORNITH_RNG_PHILOX, "unknown generator %d", s->rng);
    LOOP_TRY(ornith_top_sampler_create(c, s->temperature, s->top_p, s->top_k, s->seed, vocab, &top));
    ratio = s->accept == ORNITH_ACCEPT_RATIO;
    return ornith_top_sampler_set_rng(top, s->rng);
  }
  int next_bits(uint32_t* bits) { return ornith_top_sampler_next_bits(top, bits); }
  bool rows_are_independent() const { return top == nullptr; }
  // one row of logits -> token on the device
  int sample(const void* d_logits_row, uint32_t* d_token) {
    if (top) return ornith_top_sampler_sample(top, d_logits_row, d_token);
    return ornith_greedy_rows(ctx, d_logits_row, 1, V, d_token, nullptr);
  }
};

// prefill (src/generate.rs:90-136): everything but the last token, in chunks
inline int prefill(ornith_model* m, ornith_caches* c, const uint32_t* prompt, size_t total, size_t step,
            uint32_t* d_tok, void* d_hidden, ornith_progress_cb progress, void* user,
            size_t* processed_out) {
  size_t processed = 0;
  if (progress) progress(0, total, user);
  const size_t chunk = std::max<size_t>(1, std::min<size_t>(step, (size_t)m->max_rows));
  while (total - processed > 1) {
    const size_t n = std::min(chunk, total - processed - 1);
    LOOP_TRY(ornith_upload(m->ctx, d_tok, prompt + processed, n * 4));
    LOOP_TRY(ornith_model_forward(m, c, d_tok, (int)n, 0, d_hidden));
    LOOP_TRY(ornith_sync(m->ctx));
    processed += n;
    if (progress) progress(processed, total, user);
  }
  *processed_out = processed;
  return ORNITH_OK;
}
