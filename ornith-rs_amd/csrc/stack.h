// Models that are a list of layers (any mixer of mlstm.hip / diff_attn.hip, a dense feed-forward or
// none) around a 32-bit residual stream with pre-norms. A design's loader fills an ornith_model's
// layers; these are its registry entry's step functions.
#pragma once

#include "model.h"

size_t stack_step_bytes(const ornith_model* m, int rows);
int stack_forward(ornith_model* m, ornith_caches* cc, const uint32_t* d_tokens, int T, bool capture, void* d_hidden);
int stack_logits(ornith_model* m, const void* d_hidden, int T, void* d_logits, int dtype);
// After the layers are filled in: what each keeps, the step buffers.
int stack_finish_load(ornith_model* m);
