// The plain generation loop.
//
// Mirrors generate::{prefill, step, generate_step} (/root/reference/src/generate.rs:86-206): same
// order of model calls, same points at which a token is handed to the caller, same cache contract
// (on return the caches hold the prompt plus exactly the tokens shown to on_token). It drives any
// design of the registry.
#include "loops.h"

#define TRY LOOP_TRY

extern "C" {

int ornith_generate(ornith_model* m, ornith_caches* c, const uint32_t* prompt, size_t n_prompt,
                    const ornith_sampler* sampler, size_t max_tokens, size_t prefill_step,
                    ornith_progress_cb progress, ornith_token_cb on_token, void* user) {
  ORN_REQUIRE(m && c && prompt && on_token, "generate: null argument");
  ORN_REQUIRE(n_prompt >= 1, "generate_step needs a prompt");
  // caches whose capacity has been fixed (ornith_caches_set_growable(c, 0)): refuse a run that
  // cannot finish before any token has been handed out; growable ones grow as the rows arrive
  ORN_REQUIRE(caches_fit(c, (size_t)c->offset + n_prompt + max_tokens),
              "generate: %d cached + %zu prompt + %zu new tokens exceed cache capacity %d", c->offset, n_prompt,
              max_tokens, c->capacity);
  ornith_ctx* ctx = m->ctx;
  const size_t H = m->cfg.hidden_size, V = m->cfg.vocab_size, R = m->max_rows, hs = ornith_dtype_size(m->act_dtype);
  LoopSampler smp;
  TRY(smp.init(ctx, sampler, (int)V));
  Bufs b(ctx);
  uint32_t *d_tok, *d_out;
  void *d_hidden, *d_logits;
  TRY(b.get(R * 4, (void**)&d_tok));
  TRY(b.get(4, (void**)&d_out));
  TRY(b.get(R * H * hs, &d_hidden));
  TRY(b.get(V * 2, &d_logits));

  size_t processed = 0;
  TRY(prefill(m, c, prompt, n_prompt, prefill_step, d_tok, d_hidden, progress, user, &processed));
  // step(): run the n tokens in d_tok and sample from the last position; the one wait of the
  // step is the read-back of the sampled id
  auto step = [&](const uint32_t* d_in, size_t n, uint32_t* y) -> int {
    TRY(ornith_model_forward(m, c, d_in, (int)n, 0, d_hidden));
    TRY(ornith_model_logits(m, (char*)d_hidden + (n - 1) * H * hs, 1, d_logits));
    TRY(smp.sample(d_logits, d_out));
    return ornith_download(ctx, y, d_out, 4);
  };
  uint32_t y = 0;
  TRY(ornith_upload(ctx, d_tok, prompt + processed, (n_prompt - processed) * 4));
  TRY(step(d_tok, n_prompt - processed, &y));
  if (progress) progress(n_prompt, n_prompt, user);
  size_t n = 0;
  for (;;) {
    if (n == max_tokens) return ORNITH_OK;
    uint32_t next = 0;
    // the token just sampled is fed back from where it lies on the device: the forward
    // reads it in its first launch, the sampler overwrites it in the step's last
    TRY(step(d_out, 1, &next));
    if (!on_token(y, user)) return ORNITH_OK;
    y = next;
    ++n;
  }
}
}  // extern "C"
