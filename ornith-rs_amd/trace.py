"""Trace replay: given token ids through a model, step by step; the logits at chosen places go to files.

    bin/trace_run --model DIR --dtype bfloat16|float32 --out DIR --max-tokens N

DIR holds config.json and model.safetensors (or shards and their index); config.json picks the design.
Standard input holds a step a line, as JSON:

    {"step": 3, "entries": [{"id": "x", "tokens": [11, 4], "want": [1]}], "end": ["x"]}

"tokens" continue request "x"; "want" are indexes into them, and the float32 logits at those go to
<out>/<step>.f32, row after row; "end" names requests that need their caches no more. A finished step is
reported as `done <step>` on standard output. Nothing is sampled.

It drives the library's own step function and caches, one request after the other: a request's caches are
taken from a pool at its first tokens, reset, and returned to the pool at its end."""
import argparse
import json
import os
import sys

import numpy as np


def _library(model_dir):
    """Binds the library: the built one, or one compiled now from what the model's design needs."""
    import importlib
    pkg = importlib.import_module("ornith-rs_amd")
    build = importlib.import_module("ornith-rs_amd.build")
    with open(os.path.join(model_dir, "config.json")) as f:
        design = json.load(f).get("architecture")
    pkg.LIB_PATH = build.ensure(design)
    return pkg


class Replay:
    ROWS = 2048  # rows a forward call carries at most; longer portions take several calls

    def __init__(self, orn, model_dir, act_dtype, max_tokens):
        self.orn, self.max_tokens = orn, max_tokens
        self.ctx = orn.Ctx(0)
        self.ws = orn.WeightStore.open(self.ctx, model_dir)
        self.model = orn.TextModel.open(self.ctx, self.ws, model_dir, act_dtype)
        self.rows = max(16, min(self.ROWS, max_tokens))
        self.model.set_max_rows(self.rows)
        info = self.model.info
        self.V, self.row_bytes = info.vocab_size, info.hidden_size * (4 if info.act_dtype == orn.F32 else 2)
        self.tokens = self.ctx.alloc(self.rows * 4)
        self.hidden = self.ctx.alloc(self.rows * self.row_bytes)
        self.wanted = self.ctx.alloc(self.rows * self.row_bytes)
        self.logits, self.logit_rows = None, 0
        self.live, self.free = {}, []

    def caches_of(self, rid):
        c = self.live.get(rid)
        if c is None:
            if self.free:
                c = self.free.pop()
                c.reset()
            else:
                c = self.model.make_cache(max(1, self.max_tokens), 1)
            self.live[rid] = c
        return c

    def end(self, rid):
        c = self.live.pop(rid, None)
        if c is not None:
            self.free.append(c)

    def logits_of(self, places):
        """float32 logits [len(places), V] of these rows of the last forward."""
        orn, n = self.orn, len(places)
        if n > self.logit_rows:
            if self.logits:
                self.logits.free()
            self.logits, self.logit_rows = self.ctx.alloc(n * self.V * 4), n
        src = self.hidden
        if places != list(range(n)):
            for i, p in enumerate(places):
                _copy_row(orn, self.ctx, self.wanted, i, self.hidden, p, self.row_bytes)
            src = self.wanted
        self.model.logits_f32_on_device(src, n, self.logits)
        return self.logits.download(np.float32, (n, self.V))

    def feed(self, rid, tokens, want):
        """A request's next tokens -> the logits at `want`, in its order."""
        caches, rows = self.caches_of(rid), {}
        for at in range(0, len(tokens), self.rows):
            part = np.asarray(tokens[at:at + self.rows], dtype=np.uint32)
            self.tokens.upload(part)
            self.model.forward_on_device(caches, self.tokens, len(part), self.hidden)
            places = sorted({w - at for w in want if at <= w < at + len(part)})
            if places:
                rows.update(zip((p + at for p in places), self.logits_of(places)))
        return [rows[w] for w in want]


def _copy_row(orn, ctx, dst, i, src, j, nbytes):
    import ctypes as C
    orn._check(orn.lib().ornith_copy(ctx.h, C.c_void_p(dst.ptr.value + i * nbytes), C.c_void_p(src.ptr.value + j * nbytes),
                                     C.c_size_t(nbytes)), "copy")


def main(argv=None):
    ap = argparse.ArgumentParser(prog="trace_run", description=__doc__, formatter_class=argparse.RawDescriptionHelpFormatter)
    ap.add_argument("--model", required=True, help="folder with config.json and the weights")
    ap.add_argument("--dtype", choices=("bfloat16", "float32"), default="bfloat16")
    ap.add_argument("--out", required=True, help="folder for the logits")
    ap.add_argument("--max-tokens", type=int, default=4096, help="tokens the caches are laid out for")
    a = ap.parse_args(argv)
    orn = _library(a.model)
    try:
        replay = Replay(orn, a.model, orn.F32 if a.dtype == "float32" else orn.BF16, a.max_tokens)
    except orn.OrnithError as e:
        print(f"trace_run: {e}", file=sys.stderr)
        return 3 if a.dtype == "float32" and "runs in bf16 only" in str(e) else 1
    for line in sys.stdin:
        if not line.strip():
            continue
        step = json.loads(line)
        rows = []
        for e in step["entries"]:
            rows += replay.feed(e["id"], e["tokens"], e.get("want", []))
        if rows:
            np.stack(rows).astype("<f4").tofile(os.path.join(a.out, f"{step['step']}.f32"))
        for rid in step.get("end", []):
            replay.end(rid)
        print(f"done {step['step']}", flush=True)
    return 0
