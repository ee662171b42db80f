"""Benchmark of the speculative decode step on one MI355X.

    python bench.py [--gpus 1] [--steps K] [--warmup W] [--tokens 200] [--depth 1]

Workload (the configuration the metric is quoted on): a seeded,
random-init Qwen3.5-35B-A3B-shaped model (40 layers = 30 gated-delta + 10 full attention,
256-expert top-8 MoE + shared expert, Q4_K/Q6_K/8-bit mix, vocab 248320, one-layer bf16
MTP head, FR-Spec draft vocabulary of 32768 ids), 51-token seeded prompt, greedy depth-1
MTP decode of 200 tokens, whose output must be byte-identical to plain greedy decode.
A "step" is one such 200-token generation; the timed region starts when the prompt has
been consumed and its last position sampled from (weights, caches and prompt state are
resident in HBM) and `value` is generated tokens per second.

`value` is a FLOOR: random-init weights accept no draft, so every cycle pays a two-row verify
plus a draft for one token. The same line carries plain greedy decode and the forced-acceptance
ceilings (every draft accepted) beside it.

Also measured in the same run and printed on the same JSON line:
  roofline      the expert gather-GEMV as the model runs it: the up launch (routing made in its
                head, gate + up + swiglu) and the down launch (down + combine) of the MoE block,
                back to back over all 40 layers' resident weights with the router's own picks, at
                verify width 2: algorithmic bytes (distinct routed experts + the shared one, three
                matrices each, + activations) over the pair's average duration from HIP events on
                the library's stream, against 8 TB/s. `by_width` repeats it at T = 1, 2, 4 with the
                number of distinct experts; `standalone_up` is the up kernel alone with the expert
                ids given (no routing head).
  per_config    BASELINE configs 1-3: the 512x2048 Q4_K mat-vec, one MoE block at T = 1, 2, 4, one
                gated-delta layer at T = 2 with per-token snapshots, each with the oracle's time on
                the host cores
  cpu_baseline  the CPU oracle running the same loop on the host cores (bounded sample); the only
                part of this script that loads anything under oracle/
"""
import argparse
import ctypes as C
import importlib
import json
import os
import sys
import time

ROOT = os.path.dirname(os.path.abspath(__file__))
sys.path.insert(0, ROOT)
sys.path.insert(0, os.path.join(ROOT, "tests"))

HBM_PEAK_GBS = 8000.0
EXPERT_BYTES = 2 * 589_824 + 860_160       # gate + up (Q4_K 512x2048) + down (Q6_K 2048x512)

# HBM bytes per launch from two `rocprofv3 --pmc` runs of `bench.py --roofline-only` (FETCH_SIZE,
# then WRITE_SIZE, KiB per dispatch) recorded in profiles/moe_up_T2_pmc.md, each scaled by what
# the same counter reads for a 256 MiB device copy (fetch x 2.0, write x 1.0): the up + down pair
# as the model launches it at verify width 2 (the router's own picks, 15.4 distinct experts on
# average; its algorithmic bytes are the `bytes_per_pair` of that loop) and the up kernel alone
# with 17 given experts. Counters cannot be read from inside this script: the figures are
# carried from that profile and labelled so.
_KIB = 1024
PROFILE_TRAFFIC = {
    "pair": {"bytes": int(round(((9565.6 + 7095.0) * 2.0 + (36.1 + 8.0) * 1.0) * _KIB)), "algorithmic_bytes": 33_557_094,
             "kernel": "moe_up_kernel<0, 64, 2, true> + moe_down_kernel<1, 8, 2> (T = 2, the router's picks)"},
    "up_alone": {"bytes": int(round((9865.3 * 2.0 + 36.0 * 1.0) * _KIB)), "algorithmic_bytes": 20_080_704,
                 "kernel": "moe_up_kernel<0, 64, 2, false> (T = 2, 17 experts)"},
    "source": "profiles/moe_up_T2_pmc.md (rocprofv3 --pmc runs of `bench.py --roofline-only`, not read in this run)"}


def log(*a):
    print(*a, file=sys.stderr, flush=True)


class _Lin:
    """A Linear held by the model, seen through the struct the library hands out."""

    def __init__(self, s):
        self.s = s


def _time_loop(ctx, fn, n, warm):
    for i in range(warm):
        fn(i)
    ctx.sync()
    ctx.timer_begin()
    for i in range(n):
        fn(i)
    return ctx.timer_end() * 1000.0 / n       # microseconds per call


def expert_roofline(orn, ctx, model, np, n_layers, T, pairs=400):
    """The expert gather-GEMV as the model runs it, at verify width T: per layer the router's
    gates are made once from seeded activations, then the up launch (softmax + top-8 in its head,
    gate + up + swiglu) and the down launch (down + combine) are timed back to back, cycling
    through every layer's resident weights so that no launch finds its experts in cache.
    Algorithmic bytes per pair: (distinct routed experts + 1) x 2,039,808 + the activation rows
    read and written (x, act twice, out)."""
    rng = np.random.default_rng(123)
    H, I, E, k = 2048, 512, 256, 8
    moes = [model.moe_weights(i) for i in range(n_layers)]
    x = ctx.to_device(orn.f32_to_bf16(rng.standard_normal((T, H)).astype(np.float32)))
    gates = [ctx.alloc(T * E * 2) for _ in moes]
    egate = ctx.alloc(T * 2)
    inds, scores = ctx.alloc(T * k * 4), ctx.alloc(T * k * 2)
    act, out = ctx.alloc((T * k + T) * I * 2), ctx.alloc(T * H * 2)
    U = []
    for w, g in zip(moes, gates):
        ctx.linear_matmul(_Lin(w.router), x, T, g)
        ctx.linear_matmul(_Lin(w.sh_egate), x, T, egate)
        orn.moe_experts_from_gates(ctx, w, x, T, g, egate, inds, scores, act, out)
        U.append(len(np.unique(inds.download(np.uint32, (T * k,)))))
    us = _time_loop(ctx, lambda i: orn.moe_experts_from_gates(ctx, moes[i % n_layers], x, T, gates[i % n_layers], egate,
                                                              inds, scores, act, out), pairs, n_layers)
    u_mean = float(np.mean(U))
    acts = T * H * 2 + 2 * (T * k + T) * I * 2 + T * H * 2
    nbytes = (u_mean + 1) * EXPERT_BYTES + acts
    # the up kernel alone with the ids given (no routing head): the figure earlier reports carried
    ids = np.concatenate([rng.permutation(E)[:k] for _ in range(T)]).astype(np.uint32)
    d_ids = ctx.to_device(ids)
    us_up = _time_loop(ctx, lambda i: orn.moe_experts(ctx, moes[i % n_layers], x, T, d_ids, scores, egate, act, out, 1),
                       pairs, n_layers)
    up_bytes = (len(np.unique(ids)) + 1) * 2 * 589_824 + T * H * 2 + (T * k + T) * I * 2 + T * k * 4
    for b in [x, egate, inds, scores, act, out, d_ids] + gates:
        b.free()
    ach = nbytes / (us * 1e-6) / 1e9
    return {"verify_width": T, "distinct_experts_mean": round(u_mean, 2), "us_per_pair": round(us, 3),
            "bytes_per_pair": int(nbytes), "achieved": round(ach, 1), "frac": round(ach / HBM_PEAK_GBS, 4),
            "standalone_up": {"us_per_launch": round(us_up, 3), "bytes_per_launch": int(up_bytes),
                              "achieved": round(up_bytes / (us_up * 1e-6) / 1e9, 1),
                              "frac": round(up_bytes / (us_up * 1e-6) / 1e9 / HBM_PEAK_GBS, 4)}}


def expert_overlap(orn, ctx, model, np, n_layers, cases=("distinct", "same8"), widths=(2, 4), pairs=400):
    """Verify rows of real text share experts; random-init routing does not (U = 15.4 of 16 at
    T = 2). This leg gives the up + down pair routing in which all T tokens pick the same 8
    experts (`same8`) beside routing with 8 T distinct ones (`distinct`), ids given, cycling the
    layers' resident weights so that nothing is warm from an earlier launch. The kernels take a
    (token, expert) row per workgroup column, but a grid x of 64 puts the workgroups that read
    the same weight rows for different tokens on the same die, so the second token's reads are
    L2 hits: `bytes_distinct` is what memory has to deliver."""
    rng = np.random.default_rng(321)
    H, I, E, k = 2048, 512, 256, 8
    moes = [model.moe_weights(i) for i in range(n_layers)]
    rows = []
    for T in widths:
        x = ctx.to_device(orn.f32_to_bf16(rng.standard_normal((T, H)).astype(np.float32)))
        scores = ctx.to_device(orn.f32_to_bf16((rng.random((T, k)) + 0.1).astype(np.float32)))
        egate = ctx.to_device(orn.f32_to_bf16(rng.standard_normal((T,)).astype(np.float32)))
        act, out = ctx.alloc((T * k + T) * I * 2), ctx.alloc(T * H * 2)
        for case in cases:
            ids = []
            for _ in range(n_layers):
                if case == "same8":
                    v = np.tile(rng.permutation(E)[:k], T)
                else:
                    v = rng.permutation(E)[:k * T]
                ids.append(ctx.to_device(v.astype(np.uint32)))
            us = _time_loop(ctx, lambda i: orn.moe_experts(ctx, moes[i % n_layers], x, T, ids[i % n_layers], scores, egate,
                                                           act, out, 3), pairs, n_layers)
            U = k if case == "same8" else k * T
            nbytes = (U + 1) * EXPERT_BYTES + T * H * 2 * 2 + 2 * (T * k + T) * I * 2
            rows.append({"verify_width": T, "routing": case, "distinct_experts": U, "us_per_pair": round(us, 3),
                         "bytes_distinct": int(nbytes), "GB_s": round(nbytes / (us * 1e-6) / 1e9, 1)})
            for b in ids:
                b.free()
        for b in (x, scores, egate, act, out):
            b.free()
    return rows


def per_config(orn, ctx, np, with_cpu):
    """BASELINE configs 1-3 on their own seeded tensors: GPU time from HIP events over chained
    launches; CPU time of the oracle's restatement of the same operator (best of 5)."""
    import util
    res = {}

    def cpu_us(fn, reps=5):
        best = 1e30
        for _ in range(reps):
            t0 = time.perf_counter()
            fn()
            best = min(best, time.perf_counter() - t0)
        return round(best * 1e6, 1)

    # ---- config 1: Q4_K mat-vec 512 x 2048, fp32 activations in and out
    rng = np.random.default_rng(1)
    O, K = 512, 2048
    t = util.make_q4k(rng, 1, O, K)
    w = orn.KMatrix(ctx, orn.Q4K, *t, 1, O, K)
    xf = rng.standard_normal((1, K)).astype(np.float32)
    dx, dy = ctx.to_device(xf), ctx.alloc(O * 4)
    us = _time_loop(ctx, lambda i: ctx.kq_qmv(w, dx, orn.F32, 1, dy, orn.F32), 2000, 100)
    nbytes = 589_824 + 8_192 + 2_048
    c1 = {"workload": "Q4_K dequant mat-vec 512x2048, fp32 x [1,2048] -> fp32 y [1,512], 2000 chained launches",
          "us_per_launch": round(us, 3), "algorithmic_bytes": nbytes, "GB_s": round(nbytes / (us * 1e-6) / 1e9, 1)}
    if with_cpu:
        got = dy.download(np.float32, (1, O))
        want64 = util.orc_matvec_f64(util.Q4K, *t, O, K, xf)
        c1["max_abs_err_vs_f64"] = float(np.max(np.abs(got - want64)))
        c1["global_rel_err_vs_f64"] = util.global_rel(got, want64)
        c1["bit_exact_vs_oracle"] = bool(np.array_equal(got.view(np.uint32), util.orc_qmv(util.Q4K, *t, O, K, xf).view(np.uint32)))
        c1["cpu_us"] = cpu_us(lambda: util.orc_qmv(util.Q4K, *t, O, K, xf))
    for b in (dx, dy):
        b.free()
    w.free()
    res["config1"] = c1

    # ---- config 2: one MoE block at T = 1, 2, 4 (four sets of weights cycled: 2.1 GB)
    rng = np.random.default_rng(2)
    moes = [util.HostMoe(rng) for _ in range(4)]
    devs = [m.dev(orn, ctx) for m in moes]
    c2 = {"workload": "one MoE block: hidden 2048, 256 experts top-8 (gate/up Q4_K, down Q6_K) + shared expert, "
                      "router Q6_K, bf16 activations; router + up + down launches", "by_width": []}
    for T in (1, 2, 4):
        xb = orn.f32_to_bf16(rng.standard_normal((T, 2048)).astype(np.float32))
        dxb, dout = ctx.to_device(xb), ctx.alloc(T * 2048 * 2)
        di, ds = ctx.alloc(T * 8 * 4), ctx.alloc(T * 8 * 2)
        ctx.moe_block(devs[0], dxb, T, dout, di, ds)
        inds = di.download(np.uint32, (T, 8))
        U = len(np.unique(inds))
        us = _time_loop(ctx, lambda i: ctx.moe_block(devs[i % 4], dxb, T, dout), 400, 8)
        nbytes = (U + 1) * EXPERT_BYTES + 430_080 + 2_208 + T * 2048 * 2 * 2 + 2 * 9 * T * 1024
        e = {"T": T, "distinct_experts": U, "us_per_block": round(us, 3), "algorithmic_bytes": int(nbytes),
             "GB_s": round(nbytes / (us * 1e-6) / 1e9, 1), "frac_of_hbm_peak": round(nbytes / (us * 1e-6) / 1e9 / HBM_PEAK_GBS, 4)}
        if with_cpu:
            _, oinds, _, _ = util.orc_moe_block(moes[0], xb, T)
            e["expert_indices_bit_exact"] = bool(np.array_equal(oinds, inds))
            e["cpu_us"] = cpu_us(lambda: util.orc_moe_block(moes[0], xb, T), reps=3)
        c2["by_width"].append(e)
        for b in (dxb, dout, di, ds):
            b.free()
    for m in moes:
        m.free()
    res["config2"] = c2

    # ---- config 3: one gated-delta layer at T = 2 with per-token snapshots (rollback is a cursor move)
    rng = np.random.default_rng(3)
    H, Hk, Hv, D = 2048, 16, 32, 8192
    T = 2
    lin = {n: util.HostLinear.kq(rng, util.Q4K, o, k) for n, (o, k) in
           (("qkv", (D, H)), ("z", (4096, H)), ("out", (H, 4096)))}
    dl = {n: l.dev(orn, ctx) for n, l in lin.items()}
    wa, wb = util.HostLinear.dense(rng, Hv, H), util.HostLinear.dense(rng, Hv, H)
    bf = lambda shape, std=1.0: orn.f32_to_bf16((rng.standard_normal(shape) * std).astype(np.float32))
    host = dict(xn=bf((T, H)), conv=bf((3, D)), cw=bf((D, 4), 0.5), a_log=bf((Hv,), 0.5), dt=bf((Hv,), 0.5),
                nw=bf((128,)), S0=(rng.standard_normal((Hv, 128, 128)) * 0.1).astype(np.float32))
    d = {n: ctx.to_device(a) for n, a in host.items()}
    d["wa"], d["wb"] = ctx.to_device(wa.w), ctx.to_device(wb.w)
    qkv, z = ctx.alloc(T * D * 2), ctx.alloc(T * 4096 * 2)
    snaps, ci, gated, r = ctx.alloc(T * Hv * 128 * 128 * 4), ctx.alloc((3 + T) * D * 2), ctx.alloc(T * 4096 * 2), ctx.alloc(T * H * 2)

    def layer(i):
        ctx.linear_matmul_multi([dl["qkv"], dl["z"]], d["xn"], T, [qkv, z])
        orn.gdn_step(ctx, d["conv"], qkv, d["cw"], d["wa"], d["wb"], d["xn"], H, d["a_log"], d["dt"], T, 4, Hk, 128, Hv,
                     128, d["S0"], snaps, True, d["nw"], z, ci, gated)
        ctx.linear_matmul(dl["out"], gated, T, r)

    us = _time_loop(ctx, layer, 400, 8)
    wbytes = 9_437_184 + 4_718_592 + 4_718_592 + 2 * 131_072 + 65_536
    state = 2_097_152 * (1 + T)
    c3 = {"workload": "one gated-delta layer, T = 2 verify rows with a state snapshot per row: in_proj qkv+z, "
                      "mixer core (a/b projections, conv, recurrence, gated norm), out_proj; 3 launches, the same "
                      "weights every call; rollback of the rejected row is a cursor move (no launch)",
          "us_per_layer": round(us, 3), "weight_bytes": wbytes, "state_bytes_moved": state,
          "GB_s": round((wbytes + state) / (us * 1e-6) / 1e9, 1)}
    if with_cpu:
        def cpu_layer():
            x32 = util.bf16_to_f32(host["xn"])
            qkv_h = util.f32_to_bf16(util.orc_qmv(util.Q4K, lin["qkv"].km.qs, lin["qkv"].km.scales, lin["qkv"].km.dm, D, H, x32, True))
            z_h = util.f32_to_bf16(util.orc_qmv(util.Q4K, lin["z"].km.qs, lin["z"].km.scales, lin["z"].km.dm, 4096, H, x32, True))
            a_h, b_h = np.empty((T, Hv), np.uint16), np.empty((T, Hv), np.uint16)
            util.oracle().orc_dense_gemv(util.p(wa.w), Hv, H, util.p(host["xn"]), T, util.p(a_h))
            util.oracle().orc_dense_gemv(util.p(wb.w), Hv, H, util.p(host["xn"]), T, util.p(b_h))
            q, k, v, beta, g, _ = util.orc_gdn_front(host["conv"], qkv_h, host["cw"], a_h, b_h, host["a_log"], host["dt"], Hk, Hv)
            y, _ = util.orc_gdn_recurrence(q, k, v, g, beta, host["S0"])
            gated_h = util.orc_rms_norm_gated(y.reshape(T * Hv, 128), host["nw"], z_h.reshape(T * Hv, 128))
            return util.f32_to_bf16(util.orc_qmv(util.Q4K, lin["out"].km.qs, lin["out"].km.scales, lin["out"].km.dm, H, 4096,
                                                 util.bf16_to_f32(gated_h.reshape(T, 4096)), True))

        want = cpu_layer()
        c3["bit_exact_vs_oracle"] = bool(np.array_equal(r.download(np.uint16, (T, H)), want))
        c3["cpu_us"] = cpu_us(cpu_layer, reps=3)
    for b in list(d.values()) + [qkv, z, snaps, ci, gated, r]:
        b.free()
    for l in dl.values():
        l.free()
    res["config3"] = c3
    return res


def cpu_baseline(synth, synth_model, np, depth, tokens, prompt):
    """The oracle's generate_step_mtp on the host cores with the benchmark's own prompt; the
    prefill (timed separately on a second state) is taken off the whole call."""
    threads = int(os.environ.get("OMP_NUM_THREADS", os.cpu_count() or 1))
    fr_ids = synth.zipf_frspec_ids(synth_model.cfg["vocab_size"], 32768, seed=1)
    fr_host = synth.prune_head(synth_model.lm_head, fr_ids)
    pre = synth.OracleRun(synth_model, 128)
    t0 = time.time()
    for i in range(0, len(prompt) - 1, 16):
        pre.forward(prompt[i:min(i + 16, len(prompt) - 1)])
    t_pre = time.time() - t0
    pre.close()
    run = synth.OracleRun(synth_model, 128)
    t0 = time.time()
    toks, st = run.mtp_generate(prompt, depth, tokens, fr_ids, fr_host, policy=1, prefill_step=16)
    dt = time.time() - t0
    run.close()
    dec = max(dt - t_pre, 1e-9)
    return {"value": round(len(toks) / dec, 4), "unit": "tok/s", "cores": threads, "kind": "port",
            "sample": f"oracle generate_step_mtp depth {depth} + FR-Spec on the {len(prompt)}-token prompt, first "
                      f"{len(toks)} tokens: whole call {dt:.1f} s, of which prefill {t_pre:.1f} s "
                      f"({int(st.cycles)} cycles, {int(st.accepted)} accepted)"}, toks


def moe_ab(orn, ctx, model, np, n_layers):
    """The MoE block (norm + router + up + down) as separate launches (fuse_moe_one = 0), as one
    launch with in-launch hand-offs (1), and as router + one up/down launch (2), on the resident
    weights of every layer in turn. Prints a JSON table."""
    lib = orn.lib()
    H = 2048
    rng = np.random.default_rng(5)
    moes = [model.moe_weights(i) for i in range(n_layers)]
    wn = ctx.to_device(orn.f32_to_bf16((1 + 0.1 * rng.standard_normal(H)).astype(np.float32)))
    rows = []
    for T in (1, 2, 4):
        res, y = (ctx.to_device(orn.f32_to_bf16(rng.standard_normal((T, H)).astype(np.float32))) for _ in range(2))
        h, nx, out = ctx.alloc(T * H * 2), ctx.alloc(T * H * 2), ctx.alloc(T * H * 2)
        ref = None
        for how in (0, 1, 2):
            orn.set_option("fuse_moe_one", how)

            def run(i):
                rc = lib.ornith_add_rms_moe_block(ctx.h, C.byref(moes[i % n_layers]), res.ptr, y.ptr, wn.ptr,
                                                  C.c_float(1e-6), T, h.ptr, nx.ptr, out.ptr)
                assert rc == 0, lib.ornith_last_error()

            us = _time_loop(ctx, run, 400, n_layers)
            run(0)
            o = out.download(np.uint16, (T, H))
            ref = o if ref is None else ref
            rows.append({"T": T, "fuse_moe_one": how, "us_per_block": round(us, 2), "identical": bool(np.array_equal(o, ref))})
        for b in (res, y, h, nx, out):
            b.free()
    orn.set_option("fuse_moe_one", 0)
    print(json.dumps({"moe_block_launch_structure": rows}), flush=True)


def warm_cold(orn, ctx, np):
    """What a mat-vec gains when its weights were read just before by another kernel (they then
    sit in the memory-side cache, not in the L2 of the die that needs them), against weights
    nobody read (cycling over > 600 MB of copies) and against one matrix re-used by every launch
    (warm in its own dies' L2). The read before is `ornith_copy` of the code bytes; the setting
    `other` runs the same copy on a matrix that is not used next, so `other` - `touch` is the gain
    and `none` shows what the copy itself costs in this loop. Prints a JSON table."""
    import util
    rng = np.random.default_rng(0)
    scratch = ctx.alloc(64 << 20)
    rows = []
    for name, kind, O, K in (("in_proj 12288x2048 Q4_K", util.Q4K, 12288, 2048), ("out_proj 2048x4096 Q4_K", util.Q4K, 2048, 4096),
                             ("q_proj 8192x2048 Q6_K", util.Q6K, 8192, 2048)):
        t = util.make_kq(kind, rng, 1, O, K)
        ncopy = int(600e6 // sum(a.nbytes for a in t)) + 1
        mats = [orn.KMatrix(ctx, kind, *t, 1, O, K) for _ in range(ncopy)]
        qbytes = t[0].nbytes
        for M in (1, 2):
            x = ctx.to_device(util.bf16_normal(rng, (M, K)))
            y = ctx.alloc(M * O * 2)

            def run(i, mode):
                m = mats[0] if mode == "same" else mats[i % ncopy]
                if mode == "touch":
                    ctx.copy(scratch, m.bufs[0], qbytes)
                elif mode == "other":
                    ctx.copy(scratch, mats[(i + ncopy // 2) % ncopy].bufs[0], qbytes)
                ctx.kq_qmv(m, x, orn.BF16, M, y, orn.BF16)

            row = {"matrix": name, "M": M}
            for mode in ("same", "none", "other", "touch"):
                row[mode + "_us"] = round(_time_loop(ctx, lambda i: run(i, mode), 600, 50), 2)
            rows.append(row)
            x.free(); y.free()
        for m in mats:
            m.free()
    print(json.dumps({"matvec_warm_cold": rows}), flush=True)


def ceiling(orn, ctx, np):
    """What the machine allows a decode launch, measured with the library's probe kernels
    (csrc/probe.hip): the cost of a launch that does nothing, of launches of the expert kernels'
    shapes that only stream their bytes (cold: cycling over > 1 GiB), of a long read, where
    workgroups land, and how long a word stored by one workgroup takes to reach another on the
    same die and on another. Prints one JSON object."""
    lib = orn.lib()
    res = {}
    sink = ctx.alloc(256)

    def probe(rc, what):
        if rc != 0:
            raise orn.OrnithError(f"{what}: {lib.ornith_last_error().decode()}")

    # -- launches that do nothing, back to back. The host enqueues 1000 launches per call: if
    #    the figure does not grow with the grid it is the host's enqueue rate, not the device's.
    rows = []
    for wgs, thr, args_ in ((1, 64, 0), (1152, 256, 0), (1152, 256, 1), (512, 576, 1)):
        probe(lib.ornith_probe_empty(ctx.h, wgs, thr, args_, 200), "probe_empty")
        ctx.sync()
        ctx.timer_begin()
        probe(lib.ornith_probe_empty(ctx.h, wgs, thr, args_, 2000), "probe_empty")
        us = ctx.timer_end() * 1000.0 / 2000
        ms = C.c_float()
        probe(lib.ornith_probe_empty_graph(ctx.h, wgs, thr, args_, 2000, C.byref(ms)), "probe_empty_graph")
        rows.append({"workgroups": wgs, "threads": thr, "argument_block": bool(args_), "us_per_launch": round(us, 2),
                     "us_per_launch_in_a_graph": round(ms.value * 1000.0 / 2000, 2)})
    res["empty_launch"] = rows

    # -- launches of the expert kernels' shapes with the arithmetic taken out
    big = 2 << 30
    buf = ctx.alloc(big)
    lib.ornith_memset(ctx.h, buf.ptr, 1, C.c_size_t(big))
    rows = []
    shapes = (("expert up at T=2: 1152 x 256 threads, 4 x 16 B a thread, contiguous 4 KB a wavefront (18.9 MB)", 1152, 4, 1024),
              ("expert up at T=2, a wavefront's four pieces 1152 B apart as Q4_K rows lie (18.9 MB)", 1152, 4, 1152),
              ("expert down at T=2: 512 x 256 threads, 7 x 16 B a thread (14.7 MB)", 512, 7, 1024),
              ("expert up at T=1: 576 workgroups (9.4 MB)", 576, 4, 1024),
              ("one 4 KB piece a wavefront over 4608 workgroups (75 MB)", 4608, 4, 1024),
              ("lm_head-sized: 17,460 workgroups x 16 KB (286 MB)", 17460, 4, 1024))
    for name, wgs, per, stride in shapes:
        nbytes = wgs * 256 * per * 16
        n = 400 if nbytes < (64 << 20) else 60
        best = 1e30
        for rep in range(4):   # the first pass also warms the launch path; the best of the rest is reported
            ctx.sync()
            ctx.timer_begin()
            probe(lib.ornith_probe_stream(ctx.h, buf.ptr, C.c_size_t(big), wgs, per, C.c_size_t(stride), sink.ptr, n),
                  "probe_stream")
            us = ctx.timer_end() * 1000.0 / n
            if rep:
                best = min(best, us)
        rows.append({"shape": name, "bytes": nbytes, "us_per_launch": round(best, 2),
                     "GB_s": round(nbytes / (best * 1e-6) / 1e9, 1), "frac_of_8TBs": round(nbytes / (best * 1e-6) / 8e12, 3)})
    res["stream_only_launch"] = rows

    # -- one long read
    rows = []
    for mib in (64, 256, 1024, 2048):
        n = mib << 20
        us = _time_loop(ctx, lambda i: probe(lib.ornith_probe_read(ctx.h, buf.ptr, C.c_size_t(n), sink.ptr), "probe_read"), 20, 3)
        rows.append({"MiB": mib, "us": round(us, 1), "GB_s": round(n / (us * 1e-6) / 1e9, 1), "frac_of_8TBs": round(n / (us * 1e-6) / 8e12, 3)})
    res["long_read"] = rows
    buf.free()

    # -- where workgroups land
    n = 2048
    xo = ctx.alloc(n * 4)
    agree = 0
    for rep in range(20):
        probe(lib.ornith_probe_xcc(ctx.h, n, xo.ptr), "probe_xcc")
        ids = xo.download(np.uint32, (n,))
        if rep == 0:
            first = ids[:16].tolist()
            shift = int((ids[0] - 0) % 8)
        agree += int(np.array_equal(ids, (np.arange(n) + shift) % 8))
    res["workgroup_to_xcc"] = {"first_16": first, "rule": f"xcc = (workgroup + {shift}) mod 8", "launches_following_the_rule": agree, "of": 20}
    xo.free()

    # -- a word from one workgroup to another (workgroups 0 and 8 share a die, 0 and 1 do not)
    flag, out4 = ctx.alloc(4096 * 256), ctx.alloc(64)
    flag.zero()
    rows = []
    slot = 0
    for place, cons in (("same XCC", 8), ("another XCC", 1)):
        for mode, mname in ((0, "plain store, agent-scope (sc1) loads"), (1, "sc1 store, sc1 loads"), (2, "plain store, plain loads")):
            lat, xcc = [], None
            for rep in range(9):
                probe(lib.ornith_probe_handoff(ctx.h, C.c_void_p(flag.ptr.value + 256 * slot), out4.ptr, 0, cons, mode), "probe_handoff")
                slot += 1
                o = out4.download(np.int64, (4,))
                xcc = (int(o[2]), int(o[3]))
                lat.append((o[1] - o[0]) / 100.0 if o[1] else None)
            seen = [v for v in lat if v is not None]
            rows.append({"where": place, "how": mname, "xcc_ids": xcc, "seen": len(seen), "of": len(lat),
                         "us_min": round(min(seen), 2) if seen else None, "us_median": round(float(np.median(seen)), 2) if seen else None,
                         "us_max": round(max(seen), 2) if seen else None})
    res["word_between_workgroups"] = rows
    for b in (flag, out4, sink):
        b.free()

    # -- what one vector instruction costs (2048 workgroups x 256 threads x 8 chains x 4096)
    lib.ornith_probe_valu_name.restype = C.c_char_p
    dx = ctx.to_device(np.array([1e-3, 2e-3, 3e-3, 4e-3], np.float32))
    dp = ctx.to_device(np.full(4, 0x47000007, np.uint32))   # halves: f16 7.0 and the f16 subnormal 7 * 2^-24
    wgs, iters = 2048, 4096
    dout = ctx.alloc(wgs * 256 * 4)
    rows = []
    for op in range(lib.ornith_probe_valu_count()):
        best = 1e30
        for rep in range(3):
            ctx.sync()
            ctx.timer_begin()
            probe(lib.ornith_probe_valu(ctx.h, op, wgs, iters, dx.ptr, dp.ptr, dout.ptr), "probe_valu")
            ms = ctx.timer_end()
            if rep:
                best = min(best, ms)
        text = lib.ornith_probe_valu_name(op).decode()
        name = " + ".join(part.split()[0] for part in text.split("\n\t"))   # mnemonics only; a pair counts as one
        rows.append({"instruction": name, "ms": round(best, 3),
                     "T_lane_ops_s": round(wgs * 256 * iters * 8 / (best * 1e-3) / 1e12, 1)})
    res["vector_instruction_rate"] = rows

    # -- what a kernel argument costs: a struct read by a scalar load, or preloaded flat arguments
    didx = ctx.to_device(np.array([3], np.uint32))
    ddata = ctx.alloc(64 << 10)
    ddata.zero()
    wg = 512
    dst = ctx.alloc(wg * 32)
    scrub = ctx.alloc(64 << 20)
    rows = []
    for flat in (0, 1):
        acc = []
        for rep in range(6):
            scrub.zero()   # a launch of something else between two probes, as in a decode step
            probe(lib.ornith_probe_kernarg(ctx.h, flat, wg, didx.ptr, ddata.ptr, dst.ptr), "probe_kernarg")
            st = dst.download(np.int64, (wg, 4)).astype(np.float64) / 100.0
            if rep:
                acc.append([np.mean(st[:, 1] - st[:, 0]), np.mean(st[:, 2] - st[:, 1]), np.mean(st[:, 3] - st[:, 2])])
        m = np.mean(np.array(acc), axis=0)
        rows.append({"arguments": "leading flat arguments (preloaded)" if flat else "one struct (scalar load)",
                     "us_until_the_argument_is_in_a_register": round(float(m[0]), 3),
                     "us_dependent_scalar_load": round(float(m[1]), 3), "us_dependent_vector_load": round(float(m[2]), 3)})
    res["kernel_argument"] = rows
    for b in (dx, dp, dout, didx, ddata, dst, scrub):
        b.free()
    print(json.dumps({"ceiling": res}), flush=True)


def pair_marks(orn, ctx, model, np, n_layers, T):
    """Phase time stamps of the expert up + down pair as the model launches it (one launch of a
    stamped build: `ORN_EXTRA_FLAGS=-DORN_TIMING python ornith-rs_amd/build.py`): every workgroup
    stores the 100 MHz clock at its phase boundaries; printed as percentiles over the launch's
    workgroups, in us after the launch's first workgroup started."""
    lib = orn.lib()
    if not hasattr(lib, "ornith_debug_marks_up"):
        sys.exit("bench.py --pair-marks needs the stamped build: ORN_EXTRA_FLAGS=-DORN_TIMING python ornith-rs_amd/build.py")
    rng = np.random.default_rng(123)
    H, I, E, k = 2048, 512, 256, 8
    moes = [model.moe_weights(i) for i in range(n_layers)]
    x = ctx.to_device(orn.f32_to_bf16(rng.standard_normal((T, H)).astype(np.float32)))
    gates = [ctx.alloc(T * E * 2) for _ in moes]
    egate = ctx.alloc(T * 2)
    inds, scores = ctx.alloc(T * k * 4), ctx.alloc(T * k * 2)
    act, out = ctx.alloc((T * k + T) * I * 2), ctx.alloc(T * H * 2)
    for w, g in zip(moes, gates):
        ctx.linear_matmul(_Lin(w.router), x, T, g)
        ctx.linear_matmul(_Lin(w.sh_egate), x, T, egate)
    us = _time_loop(ctx, lambda i: orn.moe_experts_from_gates(ctx, moes[i % n_layers], x, T, gates[i % n_layers], egate,
                                                              inds, scores, act, out), 200, n_layers)
    orn.moe_experts_from_gates(ctx, moes[n_layers // 2], x, T, gates[n_layers // 2], egate, inds, scores, act, out)
    ctx.sync()
    up = (C.c_longlong * (2048 * 8))()
    down = (C.c_longlong * (1024 * 8))()
    lib.ornith_debug_marks_up(up)
    lib.ornith_debug_marks_down(down)
    a = np.frombuffer(up, np.int64).reshape(2048, 8).astype(np.float64)
    a = a[a[:, 4] > 0]
    d = np.frombuffer(down, np.int64).reshape(1024, 8).astype(np.float64)
    d = d[d[:, 5] > 0]
    t0, t1 = a[:, 0].min(), d[:, 0].min()

    def row(name, v, base):
        v = (v - base) / 100.0
        return {"phase": name, "min": round(float(v.min()), 2), "p10": round(float(np.percentile(v, 10)), 2),
                "median": round(float(np.median(v)), 2), "p90": round(float(np.percentile(v, 90)), 2), "max": round(float(v.max()), 2)}

    routed = a[:, 5] > 0
    res = {"verify_width": T, "us_per_pair_stamped_build": round(us, 2),
           "up": {"workgroups": len(a), "phases": [
               row("start", a[:, 0], t0), row("gates in registers (routed workgroups)", a[routed, 6], t0),
               row("routing made (routed workgroups)", a[routed, 5], t0),
               row("weight loads issued", a[:, 1], t0), row("activations loaded", a[:, 2], t0),
               row("first two rows done", a[:, 3], t0), row("end", a[:, 4], t0),
               row("shared expert's workgroups: weight loads issued", a[~routed, 1], t0),
               row("shared expert's workgroups: end", a[~routed, 4], t0)]},
           "down": {"workgroups": len(d), "starts_us_after_the_up_launch": round(float((t1 - t0) / 100.0), 2), "phases": [
               row("start", d[:, 0], t1), row("weight loads issued", d[:, 1], t1), row("activations loaded", d[:, 2], t1),
               row("sums done (wavefront 0)", d[:, 3], t1), row("after the barrier", d[:, 4], t1), row("end", d[:, 5], t1)]}}
    if hasattr(lib, "ornith_debug_marks_down_waves"):
        # per wavefront of the down launch's workgroups (j < k: routed slot j, j >= k: the shared expert)
        wv = (C.c_longlong * (1024 * 32))()
        lib.ornith_debug_marks_down_waves(wv)
        w = np.frombuffer(wv, np.int64).reshape(1024, 32).astype(np.float64)[:len(d)]
        nw = int((w[0, :16] > 0).sum())
        res["down"]["by_wavefront_median_us"] = [
            {"wavefront": j, "rows_in_registers": round(float(np.median(w[:, j] - t1) / 100.0), 2),
             "sums_done": round(float(np.median(w[:, 16 + j] - t1) / 100.0), 2)} for j in range(nw)]
    print(json.dumps({"pair_marks": res}), flush=True)


def config5(args, orn, ctx, synth, np, model, ws, cfg, dev_name):
    """sampled speculative decode at depth 3 after a long prefill. Runs the
    whole sequence twice (the second run is the one reported; the two must give the same tokens)
    and returns its figures."""
    depth, n_prompt, n_gen, cap = 3, 6621, (1 if args.prefill_only else 256), 16384
    model.set_max_rows(args.prefill_chunk)
    caches = model.make_cache(cap, depth + 1)
    head = orn.MtpHead(model, ws, cap)
    fr_ids = synth.zipf_frspec_ids(cfg["vocab_size"], 32768, seed=1)
    fr = orn.FrSpec(model, ids=fr_ids)
    rng = np.random.default_rng(6621)
    prompt = rng.integers(0, cfg["vocab_size"], n_prompt).astype(np.uint32)
    accept = orn.ACCEPT_RATIO if args.accept == "ratio" else orn.ACCEPT_EQUALITY
    gen = orn.RNG_PHILOX if args.rng == "philox" else orn.RNG_THREEFRY
    smp = orn.Sampler(1, 0.8, 0.95, 0, 2025, accept, gen)
    res = []
    for it in range(2):
        caches.reset()
        mark = {}

        def progress(done, total):
            ctx.sync()
            if done == 0:
                mark["p0"] = time.perf_counter()
            if done == total:
                mark["p1"] = time.perf_counter()

        toks, st = orn.generate_step_mtp(model, head, fr, caches, prompt, depth, n_gen, sampler=smp,
                                         prefill_step=args.prefill_chunk, policy=orn.HISTORY_COMMITTED,
                                         progress=progress)
        ctx.sync()
        t_end = time.perf_counter()
        res.append((toks, st, mark["p1"] - mark["p0"], t_end - mark["p1"]))
        log(f"config5 run {it}: prefill {res[-1][2]:.3f} s ({n_prompt / res[-1][2]:.0f} tok/s), decode "
            f"{n_gen / res[-1][3]:.1f} tok/s, {int(st.cycles)} cycles, {int(st.accepted)}/{int(st.drafted)} accepted")
    assert res[0][0] == res[1][0], "same seed, different tokens"
    toks, st, t_pre, t_dec = res[-1]
    # active weight bytes per prompt token are read once per chunk; the GEMM work is 2 flops per
    # active weight per token: projections + router + shared expert + 8 routed experts, 40 layers
    H, I = 2048, 512
    per_layer_gdn = H * (8192 + 4096) + 4096 * H
    per_layer_att = H * (8192 + 512 + 512) + 4096 * H
    per_layer_moe = H * 256 + 9 * 3 * H * I
    flops_tok = 2.0 * (30 * per_layer_gdn + 10 * per_layer_att + 40 * per_layer_moe)
    line = {"workload": f"config5: {n_prompt}-token prefill (chunks of {args.prefill_chunk}) into a {cap}-token context, "
                        f"then sampled MTP depth-{depth} + FR-Spec decode of {n_gen} tokens (temperature 0.8, top-p 0.95, "
                        f"{'probability-ratio (rejection-sampling)' if args.accept == 'ratio' else 'token-equality'} "
                        f"acceptance, seeded {'Philox4x32-10' if args.rng == 'philox' else 'threefry'} stream)",
            "prefill_s": round(t_pre, 4), "prefill_tok_s": round(n_prompt / t_pre, 1),
            "prefill_gemm_tflops": round(flops_tok * n_prompt / t_pre / 1e12, 2),
            "prefill_frac_of_bf16_mfma_peak": round(flops_tok * n_prompt / t_pre / 2.5e15, 4),
            "decode_tok_s": round(n_gen / t_dec, 2), "cycles": int(st.cycles), "drafted": int(st.drafted),
            "accepted": int(st.accepted), "accepted_tokens_per_verify_step": round(int(st.accepted) / max(1, int(st.cycles)), 4),
            "tokens_per_verify_step": round(n_gen / max(1, int(st.cycles)), 3),
            "repeatable": True, "device": dev_name, "data": "synthetic"}
    for o in (fr, head, caches):
        o.close()
    return line


# ---- a layer-list design beside the closest existing model (`--design NAME`) -------------------
MFMA_PEAK_TFLOPS = 2500.0
DESIGN_SIZES = {
    # width, mLSTM (heads, dim, vdim), attention (heads, kv_heads, dim, vdim, window, kept), ff
    # latent attention (dim, rot_dim, vdim, rank) has the attention's heads and window, retention the mLSTM's sizes
    2048: dict(mlstm=(8, 128, 256), attn=(16, 4, 64, 128, 2048, 64), latent=(128, 64, 128, 512), ff=5632),
    4096: dict(mlstm=(8, 256, 512), attn=(32, 8, 64, 128, 4096, 128), latent=(128, 64, 128, 512), ff=11008)}


def design_config(name, width, layers, vocab):
    """`layers` layers of such a model of that width, every fourth one attention, every second one
    with a feed-forward."""
    z = DESIGN_SIZES[width]
    H, d, dv = z["mlstm"]
    h, g, ad, av, win, keep = z["attn"]
    ld, lr, lv, rank = z["latent"]
    rv, out = name == "Ranavik", []
    for i in range(layers):
        if i % 4 == 3 and rv:
            mx = {"heads": h, "dim": ld, "rot_dim": lr, "vdim": lv, "kv_rank": rank, "scale": (ld + lr) ** -0.5, "mask": {"size": win},
                  "rot": {"base": 1e4, "dims": lr, "scaling": {"factor": 4.0, "original": 4096, "fast": 32.0, "slow": 1.0}}}
            lay = {"type": "latent_attention", "mixer": mx}
        elif i % 4 == 3:
            lay = {"type": "attention", "mixer": {"heads": h, "kv_heads": g, "dim": ad, "vdim": av, "diff": 0.55,
                                                  "scale": ad ** -0.5, "mask": {"size": win, "keep_first": keep},
                                                  "rot": {"base": 250000.0, "dims": ad // 2, "scaling": {"factor": 2.0}}}}
        elif rv:
            lay = {"type": "retention", "mixer": {"heads": H, "dim": d, "vdim": dv, "rot": {"base": 1e4, "dims": d},
                                                  "decay": [1 - 2.0 ** (-5 - a) for a in range(H)]}}
        else:
            lay = {"type": "mlstm", "mixer": {"heads": H, "dim": d, "vdim": dv, "gate_cap": 15.0}}
        lay["mlp"] = {"kind": "dense", "ff": z["ff"]} if i % 2 else None
        out.append(lay)
    cfg = {"architecture": name, "vocab": vocab, "width": width, "norm": {"eps": 1e-6}, "layers": out}
    return dict(cfg, residual_mult=0.7, logit_softcap=30.0) if rv else dict(cfg, embedding={"scale": 1.0})


def design_tensors(cfg, rng, np):
    """(name, bf16 bits) of every tensor of such a model, random (blocks of one normal draw)."""
    import util
    block = util.f32_to_bf16(rng.standard_normal(1 << 22).astype(np.float32))
    f32 = util.bf16_to_f32(block)

    def mat(*shape, std=1.0, mean=0.0):
        n = int(np.prod(shape))
        at = int(rng.integers(0, 1 << 20))
        src = np.resize(f32[at:], n) * np.float32(std) + np.float32(mean)
        return util.f32_to_bf16(src).reshape(shape)

    W, V = cfg["width"], cfg["vocab"]
    plain = 1.0 if cfg["architecture"] == "Ranavik" else 0.0
    yield "embed", mat(V, W)
    yield "head", mat(V, W, std=W ** -0.5)
    yield "final.norm", mat(W, std=0.1, mean=plain)
    if plain:
        yield "embed.norm", mat(W, std=0.1, mean=plain)
    for i, lay in enumerate(cfg["layers"]):
        p, m, kind = f"l{i}.", lay["mixer"], lay["type"]
        yield p + "norm1", mat(W, std=0.1, mean=plain)
        nv = m["heads"] * m["vdim"]
        if kind in ("mlstm", "retention"):
            nk = m["heads"] * m["dim"]
            for n, o in (("q", nk), ("k", nk), ("v", nv), ("g", nv)) + ((("i", m["heads"]), ("f", m["heads"])) if kind == "mlstm" else ()):
                yield p + "mix." + n, mat(o, W, std=W ** -0.5)
            if kind == "mlstm":
                yield p + "mix.i.b", mat(m["heads"], std=0.5)
                yield p + "mix.f.b", util.f32_to_bf16(np.full(m["heads"], 3.0, np.float32))
                yield p + "mix.norm", util.f32_to_bf16(np.ones(nv, np.float32))
        elif kind == "attention":
            for n, o in (("q", m["heads"] * 2 * m["dim"]), ("k", m["kv_heads"] * 2 * m["dim"]),
                         ("v", m["kv_heads"] * m["vdim"]), ("g", m["heads"])):
                yield p + "mix." + n, mat(o, W, std=W ** -0.5)
            for n in ("lq1", "lk1", "lq2", "lk2"):
                yield p + "mix." + n, mat(m["dim"], std=0.1)
        else:
            r = m["kv_rank"]
            for n, o in (("q", m["heads"] * (m["dim"] + m["rot_dim"])), ("dkv", r + m["rot_dim"]), ("g", m["heads"])):
                yield p + "mix." + n, mat(o, W, std=W ** -0.5)
            yield p + "mix.dkv.norm", mat(r, std=0.1, mean=1.0)
            yield p + "mix.uk", mat(m["heads"] * m["dim"], r, std=r ** -0.5)
            yield p + "mix.uv", mat(nv, r, std=r ** -0.5)
            yield p + "mix.sink", mat(m["heads"], std=1.0)
        yield p + "mix.o", mat(W, nv, std=0.5 * nv ** -0.5)
        if lay["mlp"]:
            ff = lay["mlp"]["ff"]
            yield p + "norm2", mat(W, std=0.1, mean=plain)
            yield p + "mlp.gate", mat(ff, W, std=W ** -0.5)
            yield p + "mlp.up", mat(ff, W, std=W ** -0.5)
            yield p + "mlp.down", mat(W, ff, std=0.5 * ff ** -0.5)


def design_model_rates(orn, ctx, np, model, vocab, ctx_len, n_gen, rows):
    """Prefill and decode rates of a model through the plain generation loop: a ctx_len-token prompt in
    calls of `rows` rows, then n_gen greedy tokens; the second of two runs."""
    model.set_max_rows(rows)
    caches = model.make_cache(ctx_len + n_gen + 16, 1)
    prompt = np.random.default_rng(5).integers(0, vocab, ctx_len).astype(np.uint32)
    out = None
    for _ in range(2):
        caches.reset()
        mark = {}

        def progress(done, total):
            ctx.sync()
            mark["p0" if done == 0 else "p1"] = time.perf_counter()

        toks = orn.generate_step(model, caches, prompt, n_gen, prefill_step=rows, progress=progress)
        ctx.sync()
        t = time.perf_counter()
        out = {"prompt": ctx_len, "prefill_tok_s": round(ctx_len / (mark["p1"] - mark["p0"]), 1),
               "decode_tok_s": round(len(toks) / (t - mark["p1"]), 1)}
    caches.close()
    return out


class KernelTable:
    """Kernels of a design beside the like kernels of another model, timed in turn on this device:
    microseconds a launch and the fraction of the roofline (HBM bytes, or matrix-core flops where those are
    the longer time). Weights are cycled through copies of > 512 MB in all, so no launch finds them cached."""

    def __init__(self, orn, ctx, np, only):
        self.orn, self.ctx, self.np, self.only = orn, ctx, np, only
        self.rng = np.random.default_rng(7)
        self.block = self.rng.standard_normal(1 << 20).astype(np.float32)
        self.res, self.garbage = [], []

    def dev(self, shape, dtype="bf16", std=1.0):
        import util
        a = self.np.resize(self.block, int(self.np.prod(shape))) * self.np.float32(std)
        b = self.ctx.to_device(util.f32_to_bf16(a) if dtype == "bf16" else a)
        self.garbage.append(b)
        return b

    def dense(self, O, K, copies):
        orn = self.orn
        return [orn.Linear(orn.LinearStruct(orn.LIN_DENSE, O, K, orn.KMatrixStruct(), self.dev((O, K), std=K ** -0.5).ptr, None,
                                            None), []) for _ in range(copies)]

    def kq(self, kind, O, K, copies):
        import util
        km = util.HostLinear.kq(self.rng, kind, O, K)
        out = [km.dev(self.orn, self.ctx) for _ in range(copies)]
        self.garbage.extend(out)
        return out

    @staticmethod
    def copies_for(nbytes):
        return max(2, min(24, int(-(-(600 << 20) // nbytes))))

    def row(self, name, us, nbytes, flops=0.0, peer=False, note=""):
        t_hbm, t_mm = nbytes / (HBM_PEAK_GBS * 1e3), flops / (MFMA_PEAK_TFLOPS * 1e6)
        r = {"kernel": name, "us": round(us, 2), "GB_s": round(nbytes / us / 1e3, 1), "roofline_frac": round(max(t_hbm,
                t_mm) / us, 4)}
        if flops:
            r["TFLOP_s"] = round(flops / us / 1e6, 1)
            r["bound"] = "mfma" if t_mm > t_hbm else "hbm"
        if note:
            r["note"] = note
        log(("    like: " if peer else "  ") + json.dumps(r))
        return r

    def pair(self, name, mine, peer, peer_name):
        self.res.append({"what": name, "design": mine, "closest": dict(peer, kernel=peer_name) if peer else None,
                         "times_as_far": round(peer["roofline_frac"] / mine["roofline_frac"], 2) if peer else None})

    def want(self, name):
        return self.only is None or any(o in name for o in self.only)

    def calls(self, fn, made):
        """fn(ctx, call) over call structures made beforehand (the host must not be what is timed)"""
        return lambda i: fn(self.ctx, made[i % len(made)])

    def t_of(self, fn, n=200, warm=20):
        return _time_loop(self.ctx, fn, n, warm)

    def done(self):
        for b in self.garbage:
            b.free()
        return self.res


def design_kernels(orn, ctx, np, width, only=None):
    """Every kernel of Pigodra at `width` beside the like kernel of the closest model that was there before
    it (the gated-delta / gated-attention hybrid) at the same width."""
    import util
    z, W = DESIGN_SIZES[width], width
    kt = KernelTable(orn, ctx, np, only)
    rng, block = kt.rng, kt.block
    dev, dense, kq, copies_for, row, pair, want, calls, t_of = (kt.dev, kt.dense, kt.kq, kt.copies_for, kt.row, kt.pair, kt.want,
                                                                kt.calls, kt.t_of)
    H, d, dv = z["mlstm"]
    nk, nv = H * d, H * dv
    h, g, ad, av, win, keep = z["attn"]
    ff = z["ff"]
    Hk, Hv = 16, 32                  # the hybrid's gated-delta heads (its kernels are made for this many channels)
    vd = Hv * 128
    D = 2 * Hk * 128 + vd

    # ---- projections into the mixers and back, decode
    for T in (1, 4):
        if want("decode projections"):
            shapes = [nk, nk, nv, nv, H, H]
            nb = sum(shapes) * W * 2
            n = copies_for(nb)
            ws = [dense(o, W, n) for o in shapes]
            x, wn = dev((T, W), "f32"), dev((W,), std=0.1)
            ys = [ctx.alloc(T * o * 4) for o in shapes]
            outs = [orn.OUT_ACT] * 4 + [orn.OUT_F32] * 2
            us = t_of(calls(orn.dense_rows, [orn.dense_call(orn.BF16, x, T, W, [w[i % n] for w in ws], ys, outs,
                    pre=orn.PRE_NORM, norm_w=wn, w_offset=1.0) for i in range(n)]))
            mine = row(f"norm + q, k, v, gates (T = {T})", us, nb + T * W * 4 + T * sum(shapes) * 2)
            nb2 = int((D + vd) * W * 0.5625)
            n2 = copies_for(nb2)
            a, b = kq(util.Q4K, D, W, n2), kq(util.Q4K, vd, W, n2)
            xb, yb, hb, nn = dev((T, W)), dev((T, W)), ctx.alloc(T * W * 2), ctx.alloc(T * W * 2)
            w1 = dev((W,))
            o1, o2 = ctx.alloc(T * D * 2), ctx.alloc(T * vd * 2)
            us = t_of(lambda i: orn.add_rms_linear_multi(ctx, [a[i % n2], b[i % n2]], xb, yb, w1, 1e-6, T, hb, nn, [o1,
                    o2]))
            pair(f"decode projections in, T = {T}", mine, row("x", us, nb2 + T * (D + vd) * 2, peer=True),
                    "add + norm + in_proj qkv, z (Q4_K)")
            n = copies_for(W * nv * 2)
            wo = dense(W, nv, n)
            o, gate, wn2, xs = dev((T, nv), "f32"), dev((T, nv)), dev((nv,)), dev((T, W), "f32")
            us = t_of(calls(orn.dense_rows, [orn.dense_call(orn.BF16, o, T, nv, [wo[i % n]], [xs], [orn.OUT_ADD],
                    pre=orn.PRE_HEADS, norm_w=wn2, gate=gate, head_dim=dv) for i in range(n)]))
            mine = row(f"head norm, gate + output projection + sum (T = {T})", us, W * nv * 2 + T * nv * 6)
            n2 = copies_for(int(W * vd * 0.5625))
            a = kq(util.Q4K, W, vd, n2)
            xo, yo = dev((T, vd)), ctx.alloc(T * W * 2)
            us = t_of(lambda i: ctx.linear_matmul(a[i % n2], xo, T, yo))
            pair(f"decode projection out, T = {T}", mine, row("x", us, int(W * vd * 0.5625), peer=True), "out_proj (Q4_K)")
            n = copies_for(2 * ff * W * 2)
            wg, wu, wd = dense(ff, W, n), dense(ff, W, n), dense(W, ff, n)
            act = ctx.alloc(T * ff * 2)
            us = t_of(calls(orn.dense_rows, [orn.dense_call(orn.BF16, x, T, W, [wg[i % n], wu[i % n]], [act, None], [0,
                    0], pre=orn.PRE_NORM, norm_w=wn, w_offset=1.0, pair_act=orn.PAIR_GELU) for i in range(n)]))
            mine = row(f"norm + gate, up + gelu (T = {T})", us, 2 * ff * W * 2)
            us2 = t_of(calls(orn.dense_rows, [orn.dense_call(orn.BF16, act, T, ff, [wd[i % n]], [xs],
                    [orn.OUT_ADD]) for i in range(n)]))
            mine2 = row(f"down + sum (T = {T})", us2, ff * W * 2)
            if W == 2048:
                moes = [util.HostMoe(rng, E=64).dev(orn, ctx) for _ in range(4)]
                xm, om, im = dev((T, W)), ctx.alloc(T * W * 2), ctx.alloc(T * 8 * 4)
                sm = ctx.alloc(T * 8 * 2)
                ctx.moe_block(moes[0], xm, T, om, im, sm)
                U = len(np.unique(im.download(np.uint32, (T * 8,))))
                us = t_of(lambda i: ctx.moe_block(moes[i % 4], xm, T, om))
                peer = row("x", us, (U + 1) * EXPERT_BYTES + 110_000, peer=True)
                both = row(f"feed-forward, both launches (T = {T})", mine["us"] + mine2["us"], 3 * ff * W * 2)
                pair(f"decode feed-forward, T = {T}", both, peer, "MoE block (router, up, down)")
            else:
                pair(f"decode feed-forward in, T = {T}", mine, None, None)
                pair(f"decode feed-forward out, T = {T}", mine2, None, None)
        if want("decode recurrence"):
            sf = orn.mlstm_state_floats(H, d, dv)
            layers = 24
            slots = [dev((T + 2, sf), "f32", 0.01) for _ in range(layers)]
            q, k, v, gi, gf, b1 = dev((T, nk)), dev((T, nk)), dev((T, nv)), dev((T, H), "f32"), dev((T, H),
                    "f32"), dev((H,))
            o = ctx.alloc(T * nv * 4)
            us = t_of(calls(orn.mlstm, [orn.mlstm_call(act=orn.BF16, q=q, k=k, v=v, gi=gi, gf=gf, bi=b1, bf=b1,
                    gate_cap=15.0, T=T, H=H, dim=d, vdim=dv,
                                          state_in=slots[i % layers].ptr.value + ((i // layers) % 2) * sf * 4, slots=slots[i % layers], n_slots=T + 2,
                                          first_slot=1 - (i // layers) % 2, snapshots=0, o=o) for i in range(2 * layers)]))
            mine = row(f"mLSTM step (T = {T})", us, 2 * sf * 4 + T * (2 * nk + nv) * 2 + T * nv * 4)
            sd = Hv * 128 * 128
            st = [dev((2, sd), "f32", 0.01) for _ in range(layers)]
            conv, qkv, cw, wa, wb, xn = dev((3, D)), dev((T, D)), dev((D, 4)), dev((Hv, W), std=0.02), dev((Hv, W),
                    std=0.02), dev((T, W))
            al, dt, nw, zz = dev((Hv,)), dev((Hv,)), dev((128,)), dev((T, vd))
            ci, gated = ctx.alloc((3 + T) * D * 2), ctx.alloc(T * vd * 2)
            us = t_of(lambda i: orn.gdn_step(ctx, conv, qkv, cw, wa, wb, xn, W, al, dt, T, 4, Hk, 128, Hv, 128,
                    st[i % layers], st[i % layers], False, nw, zz, ci, gated))
            pair(f"decode recurrence, T = {T}", mine, row("x", us,
                    2 * sd * 4 + 2 * Hv * W * 2 + T * (D + 2 * vd) * 2 + 7 * D * 2, peer=True), "gdn_step")
        if want("decode attention"):
            for ctx_len in (256, win + keep):
                caps = 24
                off = ctx_len - T
                kc, vc = [dev((g, ctx_len, 2 * ad)) for _ in range(caps)], [dev((g, ctx_len, av)) for _ in range(caps)]
                q, k, v, gt = dev((T, h * 2 * ad)), dev((T, g * 2 * ad)), dev((T, g * av)), dev((T, h), "f32")
                co, si = ctx.rope_table(ctx_len, ad // 2, 250000.0)
                out, qr = ctx.alloc(T * h * av * 2), ctx.alloc(T * h * 2 * ad * 2)
                us = t_of(calls(orn.diff_attn, [orn.diff_attn_call(act=orn.BF16, q=q, k=k, v=v, gate=gt, cos=co, sin=si,
                        rope_dims=ad // 2, table_npos=ctx_len, T=T, H=h, G=g,
                                                  dim=ad, vdim=av, offset=off, cap=ctx_len, window=win, keep_first=keep, scale=ad ** -0.5, lam=0.5, diff=0.55,
                                                  eps=1e-6, k_cache=kc[i % caps], v_cache=vc[i % caps], q_rot=qr, out=out) for i in range(caps)]))
                mine = row(f"attention, {ctx_len} keys (T = {T})", us, g * ctx_len * (2 * ad + av) * 2)
                Hq, Hkv = W // 128, max(2, W // 1024)
                kc2, vc2 = [dev((Hkv, ctx_len, 256)) for _ in range(caps)], [dev((Hkv, ctx_len, 256)) for _ in range(caps)]
                qg, kx, vx, qw = dev((T, Hq * 512)), dev((T, Hkv * 256)), dev((T, Hkv * 256)), dev((256,))
                co2, si2 = ctx.rope_table(ctx_len, 64, 1e7)
                qr2, out2 = ctx.alloc(T * Hq * 512), ctx.alloc(T * Hq * 512)
                us = t_of(lambda i: ctx.attn_decode(qg, kx, vx, qw, qw, T, Hq, Hkv, 256, 64, 1e-6, co2, si2, ctx_len, off,
                        ctx_len, 1 / 16.0, qr2,
                                                    kc2[i % caps], vc2[i % caps], out2))
                pair(f"decode attention, {ctx_len} keys, T = {T}", mine, row("x", us, Hkv * ctx_len * 1024, peer=True),
                        "attn_decode")
    # ---- prefill
    for T in (512, 4096):
        reps = dict(n=20, warm=3)
        if want("prefill GEMM"):
            shapes = [nk, nk, nv, nv, H, H]
            ws = [dense(o, W, 1)[0] for o in shapes]
            x, wn, rows_ = dev((T, W)), dev((W,), std=0.1), ctx.alloc(T * max(W, nv) * 2)
            ys = [ctx.alloc(T * o * 4) for o in shapes]
            outs = [orn.OUT_ACT] * 4 + [orn.OUT_F32] * 2
            us = t_of(calls(orn.dense_rows, [orn.dense_call(orn.BF16, x, T, W, ws, ys, outs) for i in range(1)]), **reps)
            mine = row(f"q, k, v, gates (T = {T})", us, sum(shapes) * W * 2 + T * W * 2 + T * sum(shapes) * 2,
                    2.0 * T * W * sum(shapes))
            a, b = kq(util.Q4K, D, W, 1), kq(util.Q4K, vd, W, 1)
            o1, o2 = ctx.alloc(T * D * 2), ctx.alloc(T * vd * 2)
            us = t_of(lambda i: ctx.linear_matmul_multi([a[0], b[0]], x, T, [o1, o2]), **reps)
            peer = row("x", us, int((D + vd) * W * 0.5625) + T * (D + vd + W) * 2, 2.0 * T * W * (D + vd), peer=True)
            pair(f"prefill GEMM in, T = {T}", mine, peer, "in_proj qkv, z (Q4_K)")
            wg, wu, wd = dense(ff, W, 1)[0], dense(ff, W, 1)[0], dense(W, ff, 1)[0]
            act, xs = ctx.alloc(T * ff * 2), dev((T, W), "f32")
            us = t_of(calls(orn.dense_rows, [orn.dense_call(orn.BF16, x, T, W, [wg, wu], [act, None], [0, 0],
                    pair_act=orn.PAIR_GELU) for i in range(1)]), **reps)
            pair(f"prefill GEMM gate, up + gelu, T = {T}", row(f"gate, up + gelu (T = {T})", us,
                    2 * ff * W * 2 + T * (W + ff) * 2, 4.0 * T * W * ff), peer, "in_proj qkv, z (Q4_K)")
            us = t_of(calls(orn.dense_rows, [orn.dense_call(orn.BF16, act, T, ff, [wd], [xs],
                    [orn.OUT_ADD]) for i in range(1)]), **reps)
            mine = row(f"down + sum (T = {T})", us, ff * W * 2 + T * (ff * 2 + W * 8), 2.0 * T * W * ff)
            a = kq(util.Q4K, W, vd, 1)
            xo, yo = dev((T, vd)), ctx.alloc(T * W * 2)
            us = t_of(lambda i: ctx.linear_matmul(a[0], xo, T, yo), **reps)
            pair(f"prefill GEMM down + sum, T = {T}", mine, row("x", us, int(W * vd * 0.5625) + T * (W + vd) * 2,
                    2.0 * T * W * vd, peer=True), "out_proj (Q4_K)")
        if want("prefill rows"):
            xs, wn, out = dev((T, W), "f32"), dev((W,), std=0.1), ctx.alloc(T * max(W, nv) * 2)
            us = t_of(lambda i: orn.norm_rows(ctx, xs, wn, 1.0, T, W, 1e-6, orn.BF16, out), **reps)
            mine = row(f"norm rows (T = {T})", us, T * W * 6)
            xb, h1, w1 = dev((T, W)), ctx.alloc(T * W * 2), dev((W,))
            us = t_of(lambda i: ctx.add_rms_norm(xb, xb, w1, T, W, 1e-6, h1, out), **reps)
            pair(f"prefill rows: norm, T = {T}", mine, row("x", us, T * W * 8, peer=True), "add_rms_norm")
            o, gate, wn2 = dev((T, nv), "f32"), dev((T, nv)), dev((nv,))
            us = t_of(lambda i: orn.head_norm_gate(ctx, o, wn2, gate, T, H, dv, 1e-6, orn.BF16, out), **reps)
            mine = row(f"head norm, gate (T = {T})", us, T * nv * 8)
            yb, zb, w3, o3 = dev((T * Hv, 128)), dev((T * Hv, 128)), dev((128,)), ctx.alloc(T * vd * 2)
            us = t_of(lambda i: ctx.rms_norm_gated(yb, w3, zb, T * Hv, 128, 1e-6, o3), **reps)
            pair(f"prefill rows: head norm, T = {T}", mine, row("x", us, T * vd * 6, peer=True), "rms_norm_gated")
        if want("prefill recurrence"):
            sf = orn.mlstm_state_floats(H, d, dv)
            slots = dev((2, sf), "f32", 0.01)
            q, k, v, gi, gf, b1 = dev((T, nk)), dev((T, nk)), dev((T, nv)), dev((T, H), "f32"), dev((T, H),
                    "f32"), dev((H,))
            o = ctx.alloc(T * nv * 4)
            us = t_of(calls(orn.mlstm, [orn.mlstm_call(act=orn.BF16, q=q, k=k, v=v, gi=gi, gf=gf, bi=b1, bf=b1,
                    gate_cap=15.0, T=T, H=H, dim=d, vdim=dv,
                                          state_in=slots.ptr.value + (i % 2) * sf * 4, slots=slots, n_slots=2, first_slot=1 - i % 2, snapshots=0, o=o) for i in range(2)]), **reps)
            mine = row(f"mLSTM in chunks (T = {T})", us, T * (2 * nk + nv) * 2 + T * nv * 4 + 2 * sf * 4,
                    2.0 * T * H * (2 * d * dv + 32 * (d + dv)))
            qd, kdd, vdd = dev((T, Hk * 128), std=0.09), dev((T, Hk * 128), std=0.09), dev((T, vd))
            gd = ctx.to_device(np.resize(np.abs(block) * np.float32(0.1) + np.float32(0.85), T * Hv).clip(0.5,
                    0.999).astype(np.float32))
            bd, yd, sd = dev((T, Hv), std=0.3), ctx.alloc(T * vd * 2), dev((1, Hv * 128 * 128), "f32", 0.01)
            us = t_of(lambda i: ctx.gdn_recurrence(qd, kdd, vdd, gd, bd, sd, T, Hk, Hv, 128, 128, yd, sd, False), **reps)
            pair(f"prefill recurrence, T = {T}", mine, row("x", us,
                    T * (2 * Hk * 128 + 2 * vd) * 2 + 2 * Hv * 128 * 128 * 4,
                                                           2.0 * T * Hv * (2 * 128 * 128 + 32 * 256), peer=True), "gdn_recurrence (chunked)")
        if want("prefill attention"):
            q, k, v, gt = dev((T, h * 2 * ad)), dev((T, g * 2 * ad)), dev((T, g * av)), dev((T, h), "f32")
            co, si = ctx.rope_table(T, ad // 2, 250000.0)
            kc, vc = dev((g, T, 2 * ad)), dev((g, T, av))
            out, qr = ctx.alloc(T * h * av * 2), ctx.alloc(T * h * 2 * ad * 2)
            i_ = np.arange(T)
            seen = float(np.sum(np.minimum(i_ + 1, win) + np.minimum(np.maximum(i_ - win + 1, 0), keep)))
            us = t_of(calls(orn.diff_attn, [orn.diff_attn_call(act=orn.BF16, q=q, k=k, v=v, gate=gt, cos=co, sin=si,
                    rope_dims=ad // 2, table_npos=T, T=T, H=h, G=g, dim=ad,
                                              vdim=av, offset=0, cap=T, window=win, keep_first=keep, scale=ad ** -0.5, lam=0.5, diff=0.55, eps=1e-6,
                                              k_cache=kc, v_cache=vc, q_rot=qr, out=out) for i in range(1)]), **reps)
            mine = row(f"attention (T = {T}, rotation and append included)", us,
                    T * (h * 2 * ad + g * (2 * ad + av) + h * av) * 2, 2.0 * seen * h * 2 * (ad + av))
            Hq, Hkv = W // 128, max(2, W // 1024)
            qg, kx, vx, qw = dev((T, Hq * 512)), dev((T, Hkv * 256)), dev((T, Hkv * 256)), dev((256,))
            co2, si2 = ctx.rope_table(T, 64, 1e7)
            kc2, vc2 = dev((Hkv, T, 256)), dev((Hkv, T, 256))
            qr2, out2 = ctx.alloc(T * Hq * 512), ctx.alloc(T * Hq * 512)
            us = t_of(lambda i: ctx.attn_decode(qg, kx, vx, qw, qw, T, Hq, Hkv, 256, 64, 1e-6, co2, si2, T, 0, T,
                    1 / 16.0, qr2, kc2, vc2, out2), **reps)
            full = T * (T + 1) / 2
            pair(f"prefill attention, T = {T}", mine, row("x", us, T * (Hq * 512 + 2 * Hkv * 256 + Hq * 256) * 2,
                    2.0 * full * Hq * 512, peer=True),
                 "attn_decode at prefill width (prep + attention)")
    return kt.done()


def ranavik_kernels(orn, ctx, np, width, only=None):
    """Every kernel of Ranavik at `width` beside the like kernel of Pigodra at the same width: retention beside
    the mLSTM at equal heads, latent attention beside differential attention at equal heads, value width and
    window."""
    z, W = DESIGN_SIZES[width], width
    kt = KernelTable(orn, ctx, np, only)
    dev, dense, copies_for, row, pair, want, calls, t_of = (kt.dev, kt.dense, kt.copies_for, kt.row, kt.pair, kt.want, kt.calls,
                                                            kt.t_of)
    H, d, dv = z["mlstm"]
    nk, nv = H * d, H * dv
    h, g, ad, av, win, keep = z["attn"]
    ld, lr, lv, rank = z["latent"]
    ff = z["ff"]
    B, ACT, F32, ADD = orn.BF16, orn.OUT_ACT, orn.OUT_F32, orn.OUT_ADD

    def projections(what, T, mine_shapes, peer_shapes, mine_outs, peer_outs, pre):
        """A mixer's input projections of both designs, with the norm in front at decode widths."""
        made, reps = [], {} if T < 32 else dict(n=20, warm=3)
        for shapes, outs in ((mine_shapes, mine_outs), (peer_shapes, peer_outs)):
            nb = sum(shapes) * W * 2
            n = copies_for(nb) if T < 32 else 1
            ws = [dense(o, W, n) for o in shapes]
            x, wn = dev((T, W), "f32" if pre else "bf16"), dev((W,), std=0.1)
            ys = [ctx.alloc(T * o * 4) for o in shapes]
            us = t_of(calls(orn.dense_rows, [orn.dense_call(B, x, T, W, [w[i % n] for w in ws], ys, outs,
                                                           pre=orn.PRE_NORM if pre else orn.PRE_NONE, norm_w=wn) for i in range(n)]), **reps)
            made.append(row("x", us, nb + T * W * 4 + T * sum(shapes) * 2, 2.0 * T * W * sum(shapes) if T >= 32 else 0.0,
                            peer=bool(made)))
            for b in ys:
                b.free()
        pair(f"{what}, T = {T}", made[0], made[1], "the same into its like")

    ret_in, mem_in = [nk, nk, nv, nv], [nk, nk, nv, nv, H, H]
    lat_in, dif_in = [h * (ld + lr), h, rank + lr], [h * 2 * ad, g * 2 * ad, g * av, h]
    for T in (1, 4, 512, 4096):
        if want("decode projections" if T < 32 else "prefill GEMM"):
            kind = "decode projections" if T < 32 else "prefill GEMM"
            projections(f"{kind} into retention", T, ret_in, mem_in, [ACT] * 4, [ACT] * 4 + [F32] * 2, T < 32)
            projections(f"{kind} into latent attention", T, lat_in, dif_in, [ACT, F32, F32], [ACT] * 3 + [F32], T < 32)
    for T in (1, 4):
        if want("decode projections"):
            n = copies_for(W * nv * 2)
            wo = dense(W, nv, n)
            o, gate, wn2, xs = dev((T, nv), "f32"), dev((T, nv)), dev((nv,)), dev((T, W), "f32")
            us = [t_of(calls(orn.dense_rows, [orn.dense_call(B, o, T, nv, [wo[i % n]], [xs], [ADD], pre=orn.PRE_HEADS, norm_w=w,
                                                            gate=gate, head_dim=dv, gate_act=act, add_scale=m) for i in range(n)]))
                  for w, act, m in ((None, orn.GATE_SILU, 0.7), (wn2, orn.GATE_SIGMOID, 1.0))]
            nb = W * nv * 2 + T * nv * 6
            pair(f"decode projection out, T = {T}", row("head norm, silu gate + output projection + sum", us[0], nb),
                 row("x", us[1], nb, peer=True), "head norm, gate + output projection + sum")
            n = copies_for(2 * ff * W * 2)
            wg, wu, wd = dense(ff, W, n), dense(ff, W, n), dense(W, ff, n)
            x, wn, act = dev((T, W), "f32"), dev((W,), std=0.1), ctx.alloc(T * ff * 2)
            us = [t_of(calls(orn.dense_rows, [orn.dense_call(B, x, T, W, [wg[i % n], wu[i % n]], [act, None], [0, 0], pre=orn.PRE_NORM,
                                                            norm_w=wn, pair_act=a) for i in range(n)]))
                  for a in (orn.PAIR_SILU, orn.PAIR_GELU)]
            pair(f"decode gate, up, T = {T}", row("norm + gate, up + silu", us[0], 2 * ff * W * 2),
                 row("x", us[1], 2 * ff * W * 2, peer=True), "norm + gate, up + gelu")
            ws = [dense(o, W, n) for o in ret_in]
            ys, wn2 = [ctx.alloc(T * o * 4) for o in ret_in], dev((W,), std=0.1)
            duo = [(orn.dense_call(B, x, T, W, [w[i] for w in ws], ys, [ACT] * 4, pre=orn.PRE_NORM, norm_w=wn2),
                    orn.dense_call(B, x, T, W, [wg[i], wu[i]], [act, None], [0, 0], pre=orn.PRE_NORM, norm_w=wn, pair_act=orn.PAIR_SILU))
                   for i in range(n)]
            us = [t_of(calls(orn.dense_rows_duo, duo)), t_of(lambda i: [orn.dense_rows(ctx, c) for c in duo[i % n]])]
            nb = (2 * ff + sum(ret_in)) * W * 2
            pair(f"decode projections beside gate, up, T = {T}", row("norms + q, k, v, g and gate, up + silu", us[0], nb),
                 row("x", us[1], nb, peer=True), "the same in two launches")
            us = [t_of(calls(orn.dense_rows, [orn.dense_call(B, act, T, ff, [wd[i % n]], [xs], [ADD], add_scale=m) for i in range(n)]))
                  for m in (0.7, 1.0)]
            pair(f"decode down, T = {T}", row("down + sum", us[0], ff * W * 2), row("x", us[1], ff * W * 2, peer=True), "down + sum")
        if want("decode recurrence"):
            layers = 24
            co, si = ctx.rope_table(64, d, 1e4)
            pw = ctx.alloc(H * orn.DECAY_POWERS * 4)
            orn.decay_powers(ctx, [1 - 2.0 ** (-5 - i % 8) for i in range(H)], pw)
            q, k, v, gi, gf, b1 = dev((T, nk)), dev((T, nk)), dev((T, nv)), dev((T, H), "f32"), dev((T, H), "f32"), dev((H,))
            o = ctx.alloc(T * nv * 4)
            sf = orn.retention_state_floats(H, d, dv)
            slots = [dev((T + 2, sf), "f32", 0.01) for _ in range(layers)]
            at = lambda i, sf: dict(state_in=slots[i % layers].ptr.value + ((i // layers) % 2) * sf * 4, slots=slots[i % layers],
                                    n_slots=T + 2, first_slot=1 - (i // layers) % 2, snapshots=0, o=o)
            us = t_of(calls(orn.retention, [orn.retention_call(act=B, q=q, k=k, v=v, cos=co, sin=si, rope_dims=d, table_npos=64, offset=9,
                                                              decay=pw, T=T, H=H, dim=d, vdim=dv, **at(i, sf)) for i in range(2 * layers)]))
            mine = row("retention step", us, 2 * sf * 4 + T * (2 * nk + nv) * 2 + T * nv * 4)
            sm = orn.mlstm_state_floats(H, d, dv)
            slots = [dev((T + 2, sm), "f32", 0.01) for _ in range(layers)]
            us = t_of(calls(orn.mlstm, [orn.mlstm_call(act=B, q=q, k=k, v=v, gi=gi, gf=gf, bi=b1, bf=b1, gate_cap=15.0, T=T, H=H, dim=d,
                                                      vdim=dv, **at(i, sm)) for i in range(2 * layers)]))
            pair(f"decode recurrence, T = {T}", mine, row("x", us, 2 * sm * 4 + T * (2 * nk + nv) * 2 + T * nv * 4, peer=True), "mLSTM step")

    def attention(T, ctx_len, off, caps, reps):
        """Latent attention (append, maps, sink and gate included) beside differential attention."""
        co, si = ctx.rope_table(ctx_len, lr, 1e4)
        cc, rc = [dev((ctx_len, rank)) for _ in range(caps)], [dev((ctx_len, lr)) for _ in range(caps)]
        uk, uv = dense(h * ld, rank, caps), dense(h * lv, rank, caps)
        q, down, nw, gt, sink = dev((T, h * (ld + lr))), dev((T, rank + lr), "f32"), dev((rank,)), dev((T, h), "f32"), dev((h,))
        out = ctx.alloc(T * h * max(lv, av) * 2)
        us = t_of(calls(orn.latent_attn, [orn.latent_attn_call(
            uk[i], uv[i], act=B, q=q, down=down, down_norm=nw, gate=gt, sink=sink, cos=co, sin=si, table_npos=ctx_len, T=T, H=h, dim=ld,
            rot_dim=lr, vdim=lv, rank=rank, offset=off, cap=ctx_len, window=win, scale=(ld + lr) ** -0.5, eps=1e-6, c_cache=cc[i],
            r_cache=rc[i], out=out) for i in range(caps)]), **reps)
        i_ = np.arange(off, off + T)
        seen = float(np.sum(np.minimum(i_ + 1, win)))
        maps = h * (ld + lv) * rank
        wide = T >= 32
        mine = row("latent attention", us, maps * 2 + min(ctx_len, win + T) * (rank + lr) * 2 + T * (h * (ld + lr + lv) * 2 + (rank + lr) * 4),
                   2.0 * T * maps + 2.0 * seen * h * (ld + lr + lv) if wide else 0.0)
        kc, vc = [dev((g, ctx_len, 2 * ad)) for _ in range(caps)], [dev((g, ctx_len, av)) for _ in range(caps)]
        q, k, v = dev((T, h * 2 * ad)), dev((T, g * 2 * ad)), dev((T, g * av))
        co, si = ctx.rope_table(ctx_len, ad // 2, 250000.0)
        qr = ctx.alloc(T * h * 2 * ad * 2)
        us = t_of(calls(orn.diff_attn, [orn.diff_attn_call(
            act=B, q=q, k=k, v=v, gate=gt, cos=co, sin=si, rope_dims=ad // 2, table_npos=ctx_len, T=T, H=h, G=g, dim=ad, vdim=av,
            offset=off, cap=ctx_len, window=win, keep_first=0, scale=ad ** -0.5, lam=0.5, diff=0.55, eps=1e-6, k_cache=kc[i],
            v_cache=vc[i], q_rot=qr, out=out) for i in range(caps)]), **reps)
        peer = row("x", us, g * min(ctx_len, win + T) * (2 * ad + av) * 2 + T * (h * 2 * ad + h * av) * 2,
                   2.0 * seen * h * 2 * (ad + av) if wide else 0.0, peer=True)
        pair(f"{'prefill' if wide else 'decode'} attention, {min(ctx_len, win)} keys, T = {T}", mine, peer, "differential attention")

    for T in (1, 4):
        if want("decode attention"):
            for n in (256, win + T):
                attention(T, n, n - T, 24, {})
    # ---- prefill
    for T in (512, 4096):
        reps = dict(n=20, warm=3)
        if want("prefill GEMM"):
            wg, wu = dense(ff, W, 1)[0], dense(ff, W, 1)[0]
            x, act = dev((T, W)), ctx.alloc(T * ff * 2)
            us = [t_of(calls(orn.dense_rows, [orn.dense_call(B, x, T, W, [wg, wu], [act, None], [0, 0], pair_act=a)]), **reps)
                  for a in (orn.PAIR_SILU, orn.PAIR_GELU)]
            size = (2 * ff * W * 2 + T * (W + ff) * 2, 4.0 * T * W * ff)
            pair(f"prefill GEMM gate, up, T = {T}", row("gate, up + silu", us[0], *size), row("x", us[1], *size, peer=True), "gate, up + gelu")
        if want("prefill rows"):
            o, gate, wn2, out = dev((T, nv), "f32"), dev((T, nv)), dev((nv,)), ctx.alloc(T * max(W, nv) * 4)
            us = [t_of(lambda i: orn.head_norm_gate(ctx, o, w, gate, T, H, dv, 1e-6, B, out, gate_act=a), **reps)
                  for w, a in ((None, orn.GATE_SILU), (wn2, orn.GATE_SIGMOID))]
            pair(f"prefill rows: head norm, T = {T}", row("head norm, silu gate", us[0], T * nv * 8),
                 row("x", us[1], T * nv * 8, peer=True), "head norm, gate")
            table, wn = dense(32768, W, 1)[0], dev((W,))
            ids = ctx.to_device(kt.rng.integers(0, 32768, T).astype(np.uint32))
            us = [t_of(lambda i: orn.embed_norm_rows(ctx, table, ids, T, wn, 0.0, 1e-6, out), **reps),
                  t_of(lambda i: orn.embed_rows(ctx, table, ids, T, 1.0, out), **reps)]
            pair(f"prefill rows: embedding, T = {T}", row("embedding + norm", us[0], T * W * 6), row("x", us[1], T * W * 6, peer=True),
                 "embedding")
        if want("prefill recurrence"):
            co, si = ctx.rope_table(T, d, 1e4)
            pw = ctx.alloc(H * orn.DECAY_POWERS * 4)
            orn.decay_powers(ctx, [1 - 2.0 ** (-5 - i % 8) for i in range(H)], pw)
            q, k, v, gi, gf, b1 = dev((T, nk)), dev((T, nk)), dev((T, nv)), dev((T, H), "f32"), dev((T, H), "f32"), dev((H,))
            o = ctx.alloc(T * nv * 4)
            sf, sm = orn.retention_state_floats(H, d, dv), orn.mlstm_state_floats(H, d, dv)
            slots = dev((2, sm), "f32", 0.01)
            at = lambda i, n: dict(state_in=slots.ptr.value + (i % 2) * n * 4, slots=slots, n_slots=2, first_slot=1 - i % 2, snapshots=0, o=o)
            size = (T * (2 * nk + nv) * 2 + T * nv * 4 + 2 * sf * 4, 2.0 * T * H * (2 * d * dv + 32 * (d + dv)))
            us = t_of(calls(orn.retention, [orn.retention_call(act=B, q=q, k=k, v=v, cos=co, sin=si, rope_dims=d, table_npos=T, offset=0,
                                                              decay=pw, T=T, H=H, dim=d, vdim=dv, **at(i, sf)) for i in range(2)]), **reps)
            mine = row("retention in chunks (rotation included)", us, *size)
            us = t_of(calls(orn.mlstm, [orn.mlstm_call(act=B, q=q, k=k, v=v, gi=gi, gf=gf, bi=b1, bf=b1, gate_cap=15.0, T=T, H=H, dim=d,
                                                      vdim=dv, **at(i, sm)) for i in range(2)]), **reps)
            pair(f"prefill recurrence, T = {T}", mine, row("x", us, *size, peer=True), "mLSTM in chunks")
        if want("prefill attention"):
            attention(T, T, 0, 1, reps)
    return kt.done()


def design_bench(args, orn, ctx, synth, np, dev_name):
    """`--design NAME`: prefill and decode rates of the design at layer sizes of real models (random
    weights) beside the closest other model at equal width and depth, and kernel by kernel."""
    out = {"design": args.design, "device": dev_name, "data": "synthetic", "models": [], "kernels": []}
    layers, vocab = 8, 32768
    only = args.design_kernels.split(",") if args.design_kernels else None
    kernels = {"Pigodra": design_kernels, "Ranavik": ranavik_kernels}[args.design]

    def rates(name, width):
        cfg = design_config(name, width, layers, vocab)
        ws = orn.WeightStore(ctx)
        for n, a in design_tensors(cfg, np.random.default_rng(3), np):
            ws.put(n, a, orn.DT_BF16)
        model = orn.TextModel.from_json(ctx, ws, cfg)
        r = [design_model_rates(orn, ctx, np, model, vocab, n, 128, 4096) for n in (128, 4096)], ws.stats()[1]
        model.close()
        ws.close()
        return r

    for width in (int(w) for w in args.design_widths.split(",")):
        log(f"width {width}: kernels")
        out["kernels"].append({"width": width, "rows": kernels(orn, ctx, np, width, only)})
        if args.design_no_models:
            continue
        e = {"width": width, "layers": layers}
        e["design"], e["weight_bytes"] = rates(args.design, width)
        if args.design == "Ranavik":
            e["closest"], e["closest_weight_bytes"] = rates("Pigodra", width)
        # the hybrid's stepwise kernels are made for hidden size 2048: its width there
        elif width == 2048:
            qc = dict(synth.FULL, num_hidden_layers=layers, vocab_size=vocab, num_experts=64)
            sm = synth.SynthModel(qc, seed=9, with_mtp=False, with_oracle=False)
            ws = sm.upload(orn, ctx, drop_host=True)
            model = orn.TextModel(ctx, ws, sm.text_config(orn))
            e["closest"] = [design_model_rates(orn, ctx, np, model, vocab, n, 128, 4096) for n in (128, 4096)]
            e["closest_weight_bytes"] = ws.stats()[1]
            model.close()
            ws.close()
        log(json.dumps(e))
        out["models"].append(e)
    print(json.dumps(out), flush=True)


def main():
    ap = argparse.ArgumentParser()
    ap.add_argument("--gpus", type=int, default=1)
    ap.add_argument("--steps", type=int, default=3)
    ap.add_argument("--warmup", type=int, default=1)
    ap.add_argument("--tokens", type=int, default=200)
    ap.add_argument("--depth", type=int, default=1)
    ap.add_argument("--layers", type=int, default=40, help="trunk layers (40 = the named config)")
    ap.add_argument("--cpu-tokens", type=int, default=40)
    ap.add_argument("--no-cpu", action="store_true", help="skip every leg that runs the CPU oracle")
    ap.add_argument("--config5", action="store_true",
                    help="instead of the metric's workload: BASELINE config 5 (6621-token prefill into a "
                         "16384-token context through the matrix-core path, then sampled depth-3 MTP "
                         "decode of 256 tokens, temperature 0.8, top-p 0.95); prints its own JSON line")
    ap.add_argument("--accept", choices=("ratio", "equality"), default="ratio",
                    help="with --config5: probability-ratio (rejection-sampling) acceptance, or the reference's token equality")
    ap.add_argument("--rng", choices=("philox", "threefry"), default="philox",
                    help="with --config5: the sampler's random stream")
    ap.add_argument("--prefill-chunk", type=int, default=8192,
                    help="rows per prefill call with --config5 (the reference's prefill_step_size is 2048; up to 8192 "
                         "here: by default the 6621-token prompt is one call)")
    ap.add_argument("--prefill-only", action="store_true",
                    help="with --config5: stop after the first generated token (a short run for "
                         "profiling the matrix-core prefill kernels)")
    ap.add_argument("--roofline-only", action="store_true",
                    help="only the expert-kernel timing loops plus three 256 MiB device copies "
                         "(the known-size reference for rocprofv3 --pmc FETCH_SIZE / WRITE_SIZE)")
    ap.add_argument("--overlap", choices=("distinct", "same8"), default=None,
                    help="only the expert pair under the named routing at T = 2 (all tokens on the same 8 experts, "
                         "or on 16 distinct ones), then three 256 MiB device copies: one rocprofv3 --pmc run a case")
    ap.add_argument("--moe-ab", action="store_true",
                    help="only the A/B of the MoE block's launch structure (option fuse_moe_one = 0, 1, 2)")
    ap.add_argument("--ceiling", action="store_true",
                    help="only the machine probes: empty launches, stream-only launches of the expert kernels' shapes, "
                         "a long read, the workgroup-to-die rule, the latency of a word between workgroups, the rate "
                         "of single vector instructions, the cost of a kernel argument")
    ap.add_argument("--pair-marks", action="store_true",
                    help="only the phase time stamps of the expert pair (needs the library built with -DORN_TIMING)")
    ap.add_argument("--warm-cold", action="store_true",
                    help="only the mat-vec timings on re-used, unread and just-read weights")
    ap.add_argument("--design", choices=("Pigodra", "Ranavik"), default=None,
                    help="instead of the metric's workload: prefill and decode rates of that design at layer sizes of real "
                         "models (random weights) beside the closest existing model, and every kernel of both")
    ap.add_argument("--design-widths", default="2048,4096", help="with --design: model widths, commas between them")
    ap.add_argument("--design-kernels", default="", help="with --design: only kernels whose group contains one of these words")
    ap.add_argument("--design-no-models", action="store_true", help="with --design: the kernels only")
    args = ap.parse_args()
    if args.gpus != 1:
        sys.exit("bench.py: this build runs on exactly one GPU (one process, one stream); "
                 "--gpus N with N > 1 is not supported and nothing here uses a second device.")

    import numpy as np
    import synth
    orn = importlib.import_module("ornith-rs_amd")
    ctx = orn.Ctx(0)
    dev_name, cus, mem = ctx.device_info()
    log(f"device: {dev_name}, {cus} CUs, {mem / 2**30:.0f} GiB")

    if args.ceiling:
        return ceiling(orn, ctx, np)
    if args.warm_cold:
        return warm_cold(orn, ctx, np)
    if args.design:
        return design_bench(args, orn, ctx, synth, np, dev_name)
    cfg = dict(synth.FULL, num_hidden_layers=args.layers)
    t0 = time.time()
    sm = synth.SynthModel(cfg, seed=2025)
    log(f"synthetic weights: {sm.total_bytes() / 1e9:.2f} GB generated in {time.time() - t0:.1f} s")
    t0 = time.time()
    ws = sm.upload(orn, ctx)
    log(f"uploaded in {time.time() - t0:.1f} s")
    model = orn.TextModel(ctx, ws, sm.text_config(orn))
    if args.roofline_only:
        roof = expert_roofline(orn, ctx, model, np, args.layers, T=args.depth + 1, pairs=200)
        a, b = ctx.alloc(256 << 20), ctx.alloc(256 << 20)
        for _ in range(3):
            ctx.copy(a, b, 256 << 20)
        ctx.sync()
        print(json.dumps({"roofline": roof}), flush=True)
        return
    if args.overlap:
        rows = expert_overlap(orn, ctx, model, np, args.layers, cases=(args.overlap,), widths=(2,), pairs=200)
        a, b = ctx.alloc(256 << 20), ctx.alloc(256 << 20)
        for _ in range(3):
            ctx.copy(a, b, 256 << 20)
        ctx.sync()
        print(json.dumps({"overlapping_routing": rows}), flush=True)
        return
    if args.moe_ab:
        return moe_ab(orn, ctx, model, np, args.layers)
    if args.pair_marks:
        return pair_marks(orn, ctx, model, np, args.layers, args.depth + 1)
    if args.config5:
        print(json.dumps(config5(args, orn, ctx, synth, np, model, ws, cfg, dev_name)), flush=True)
        return
    rng = np.random.default_rng(51)
    prompt = rng.integers(0, cfg["vocab_size"], 51).astype(np.uint32)
    cap = 4096
    caches = model.make_cache(cap, args.depth + 1)
    head = orn.MtpHead(model, ws, cap)
    fr_ids = synth.zipf_frspec_ids(cfg["vocab_size"], 32768, seed=1)
    fr = orn.FrSpec(model, ids=fr_ids)

    def timed_run(fn):
        """fn(progress) -> tokens; returns (tokens, decode seconds). Both loops report the
        prompt consumed at the same point: after its last position has been sampled from."""
        mark = {}

        def progress(done, total):
            if done == total:
                ctx.sync()
                mark["t0"] = time.perf_counter()

        out = fn(progress)
        ctx.sync()
        return out, time.perf_counter() - mark["t0"]

    # plain greedy, for the byte-identity check and as the non-speculative figure
    caches.reset()
    orn.generate_step(model, caches, prompt, 8, prefill_step=16)      # warm the shapes
    caches.reset()
    ar, ar_s = timed_run(lambda pr: orn.generate_step(model, caches, prompt, args.tokens, prefill_step=16, progress=pr))
    log(f"plain greedy: {len(ar)} tokens in {ar_s * 1e3:.1f} ms = {len(ar) / ar_s:.1f} tok/s")

    times, stats, toks = [], None, None
    for it in range(args.warmup + args.steps):
        caches.reset()
        (toks, stats), dt = timed_run(lambda pr: orn.generate_step_mtp(
            model, head, fr, caches, prompt, args.depth, args.tokens, prefill_step=16,
            policy=orn.HISTORY_COMMITTED, progress=pr))
        if toks != ar:
            sys.exit("bench.py: speculative output is NOT identical to plain greedy -- result invalid")
        if it >= args.warmup:
            times.append(dt)
        log(f"mtp depth {args.depth} run {it}: {dt * 1e3:.1f} ms, {int(stats.cycles)} cycles, "
            f"{int(stats.accepted)}/{int(stats.drafted)} accepted")
    total_s = sum(times)
    tok_s = args.tokens * len(times) / total_s

    # Forced acceptance: random-init weights accept no draft, so `value` is the floor of the
    # loop. With the known output as the drafts every draft is accepted and a cycle yields
    # depth + 1 tokens: the ceiling. The head still runs for every draft.
    forced = {}
    c2 = model.make_cache(cap, 4)
    head.force_drafts(ar)
    for d in (1, 2, 3):
        for it in range(2):   # the first run warms the shapes of this depth
            c2.reset()
            (ft, fst), fdt = timed_run(lambda pr: orn.generate_step_mtp(
                model, head, fr, c2, prompt, d, args.tokens, prefill_step=16,
                policy=orn.HISTORY_COMMITTED, progress=pr))
            if ft != ar:
                sys.exit("bench.py: forced-draft output is NOT identical to plain greedy -- result invalid")
        forced[f"depth{d}"] = {"tok_s": round(args.tokens / fdt, 1), "cycles": int(fst.cycles),
                               "accepted": int(fst.accepted), "drafted": int(fst.drafted)}
        log(f"forced acceptance depth {d}: {args.tokens / fdt:.1f} tok/s, {int(fst.cycles)} cycles, "
            f"{int(fst.accepted)}/{int(fst.drafted)} accepted")
    head.force_drafts([])
    c2.close()

    by_width = [expert_roofline(orn, ctx, model, np, args.layers, T) for T in (1, 2, 4)]
    main_w = next(w for w in by_width if w["verify_width"] == 2)
    roof = {"bound": "hbm", "achieved": main_w["achieved"], "peak": HBM_PEAK_GBS, "unit": "GB/s", "frac": main_w["frac"],
            "traffic": PROFILE_TRAFFIC["pair"]["bytes"], "traffic_from_profile": PROFILE_TRAFFIC,
            "kernel": "moe_up_kernel<Q4_K, 64, 2, routing made in the launch> + moe_down_kernel<Q6_K, 8, 2>: the expert "
                      "gather-GEMV of one MoE block as the model launches it (gate + up + swiglu, down + combine), "
                      "verify width 2, the router's own picks",
            "us_per_launch": main_w["us_per_pair"], "launches_per_unit": 2, "bytes_per_launch": main_w["bytes_per_pair"],
            "distinct_experts": main_w["distinct_experts_mean"], "verify_width": 2, "by_width": by_width,
            "overlapping_routing": expert_overlap(orn, ctx, model, np, args.layers)}
    log("roofline:", roof)

    # Whole-step figures: the algorithmic bytes one decode step has to read (and the recurrent
    # state it writes) against the time the step takes. Dense projections of 30 gated-delta and
    # 10 attention layers, per MoE block the router + (distinct routed + 1) experts, the output
    # head (all 248,320 rows of Q4_K), 2 MiB of recurrent state a gated-delta layer read once and
    # written once per row, the KV rows of a context of about 150 tokens. The depth-1 cycle adds
    # the draft: the bf16 head layer (129 MB) and the 32,768-row pruned output head.
    dense = 30 * 19_202_048 + 10 * 22_364_160
    head_full, head_pruned, mtp_layer = 286_064_640, 37_748_736, 129_000_000
    state = 30 * 2_097_152
    kv = 10 * 2 * 2 * 150 * 256 * 2

    def step_bytes(T, U):
        return dense + 40 * ((U + 1) * EXPERT_BYTES + 430_080) + head_full + state * (1 + T) + kv

    u1 = next(w for w in by_width if w["verify_width"] == 1)["distinct_experts_mean"]
    u2 = main_w["distinct_experts_mean"]
    plain_ms = ar_s / len(ar) * 1e3
    cycle_ms = total_s / len(times) / max(1, int(stats.cycles)) * 1e3
    b_plain, b_cycle = step_bytes(1, u1), step_bytes(2, u2) + mtp_layer + head_pruned
    step_roof = {"plain_greedy": {"bytes_per_token": int(b_plain), "ms_per_token": round(plain_ms, 4),
                                  "GB_s": round(b_plain / plain_ms / 1e6, 1), "frac_of_hbm_peak": round(b_plain / plain_ms / 1e6 / HBM_PEAK_GBS, 4)},
                 "mtp_depth1_cycle": {"bytes_per_cycle": int(b_cycle), "ms_per_cycle": round(cycle_ms, 4),
                                      "GB_s": round(b_cycle / cycle_ms / 1e6, 1), "frac_of_hbm_peak": round(b_cycle / cycle_ms / 1e6 / HBM_PEAK_GBS, 4)}}
    log("step_roofline:", step_roof)

    configs = per_config(orn, ctx, np, with_cpu=not args.no_cpu)
    # config 5 (sampled depth-3 decode behind a 6621-token matrix-core prefill) on the same model
    for o in (fr, head, caches):
        o.close()
    configs["config5"] = config5(args, orn, ctx, synth, np, model, ws, cfg, dev_name)
    log("per_config:", configs)

    cpu = None
    if not args.no_cpu:
        cpu, cpu_toks = cpu_baseline(synth, sm, np, args.depth, args.cpu_tokens, prompt)
        # the same tokens must have come out of the GPU
        cpu["gpu_tokens_match"] = bool(ar[:len(cpu_toks)] == cpu_toks)
        log("cpu_baseline:", cpu)

    line = {
        "metric": "decode tok/s @MTP depth 1 (1 GPU, byte-exact); expert GEMV HBM GB/s vs peak",
        "value": round(tok_s, 2), "unit": "tok/s", "n_gpus": 1, "steps": args.steps, "warmup": args.warmup,
        "ms_per_step": round(total_s / len(times) * 1e3, 3), "higher_is_better": True, "scaling": "weak",
        "vs_baseline": None, "dtype": "bf16",
        "data": "synthetic",
        "value_is": "the zero-acceptance floor of the depth-1 loop (random-init weights accept no draft: one token per "
                    "two-row verify + draft); see plain_greedy_tok_s and forced_acceptance_ceiling beside it",
        "plain_greedy_tok_s": round(len(ar) / ar_s, 2),
        "forced_acceptance_ceiling": forced,
        "config": {"workload": f"config4: greedy MTP depth-{args.depth} + FR-Spec(32768) decode of {args.tokens} tokens, "
                               f"51-token prompt, Qwen3.5-35B-A3B shape, {args.layers} layers, KV capacity {cap}",
                   "arithmetic": "bf16 activations, fp32 accumulation, Q4_K/Q6_K/int8/bf16 weights",
                   "tokens_per_step": args.tokens, "byte_identical_to_greedy": True,
                   "cycles": int(stats.cycles), "accepted": int(stats.accepted), "drafted": int(stats.drafted),
                   "weights_GB": round(ws.stats()[1] / 1e9, 2), "device": dev_name},
        "roofline": roof,
        "step_roofline": step_roof,
        "per_config": configs,
        "cpu_baseline": cpu,
    }
    print(json.dumps(line), flush=True)


if __name__ == "__main__":
    main()
