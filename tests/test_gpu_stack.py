"""GPU: the mechanisms of the layer-list designs, each alone, against float64 (tests/ref_stack.py): dense
projections with their prologues and tails, the mLSTM memory, differential attention. In 32-bit the
bound is a few fp32 roundings; in bf16 the inputs are bf16 numbers in the reference too and the bound is
the output's rounding plus the noise of two bf16 parts."""
import numpy as np
import pytest

import ref_stack as R
import util

pytestmark = pytest.mark.gpu


def _bf(a):
    return util.bf16_to_f32(util.f32_to_bf16(np.asarray(a, np.float32)))


def _dev(ctx, a, act):
    """An activation array on the device (values must be bf16 numbers when act is bf16)."""
    a = np.asarray(a, np.float32)
    return ctx.to_device(a if act == 0 else util.f32_to_bf16(a))


def _get(buf, shape, act):
    return buf.download(np.float32, shape) if act == 0 else util.bf16_to_f32(buf.download(np.uint16, shape))


def _close(got, want, act, what, slack=1.0):
    """fp32: 3e-6 of the largest magnitude around; bf16: half an ulp of the value (2^-8) and 1 % of the rms."""
    want = np.asarray(want, np.float64)
    rms = np.sqrt(np.mean(want ** 2)) + 1e-30
    bound = slack * (3e-6 * (np.abs(want) + 3 * rms) if act == 0 else 2.0 ** -8 * np.abs(want) + 1e-2 * rms)
    err = np.abs(got - want)
    assert np.all(np.isfinite(got)) and np.all(err <= bound), (what, float(err.max()), float((err / bound).max()),
            float(rms))


@pytest.mark.parametrize("act", [0, 1])
@pytest.mark.parametrize("M,K", [(1, 96), (2, 200), (3, 90), (5, 1032), (33, 200), (130, 96), (200, 264), (37, 91), (1,
        9000), (2, 4104)])
def test_dense_rows(orn, ctx, act, M, K):
    """All prologues and tails at decode and GEMM widths; widths that are no multiple of 8, ragged
    tiles, more than one matrix, rows longer than a thread's registers hold."""
    rng = np.random.default_rng(M * 10007 + K)
    Os = [33, 8, 64, 130, 1]
    W = [_bf(rng.standard_normal((o, K)) * K ** -0.5) for o in Os]
    lins = [orn.Linear.dense(ctx, util.f32_to_bf16(w)) for w in W]
    head = K // 2 if K % 2 == 0 else K // 7
    x32 = rng.standard_normal((M, K)).astype(np.float32)
    xa = _bf(x32) if act else x32
    gate = rng.standard_normal((M, K)).astype(np.float32)
    gate = _bf(gate) if act else gate
    wn = _bf(0.3 * rng.standard_normal(K))
    rows = {orn.PRE_NONE: xa.astype(np.float64), orn.PRE_NORM: R.norm_zero_centred(x32.astype(np.float64), wn, 1e-5),
            orn.PRE_HEADS: (R.rms(x32.astype(np.float64).reshape(M, -1, head), 1e-5).reshape(M,
                    K) * wn) * R.sigmoid(gate.astype(np.float64))}
    d_x, d_g, d_wn = ctx.to_device(x32), _dev(ctx, gate, act), ctx.to_device(util.f32_to_bf16(wn))
    d_xa, d_rows = _dev(ctx, xa, act), ctx.alloc(M * K * 4)
    adt, es = (orn.F32, 4) if act == 0 else (orn.BF16, 2)
    for pre, want in rows.items():
        h = want if act == 0 else _bf(want).astype(np.float64)
        outs = [orn.OUT_ACT, orn.OUT_F32, orn.OUT_ADD, orn.OUT_ACT, orn.OUT_F32]
        base = rng.standard_normal((M, Os[2])).astype(np.float32)
        ys = [ctx.alloc(M * o * 4) for o in Os]
        ys[2].upload(base)
        orn.dense_rows(ctx, adt, d_xa if pre == orn.PRE_NONE else d_x, M, K, lins, ys, outs, pre=pre,
                       norm_w=d_wn, gate=d_g, w_offset=1.0, eps=1e-5, head_dim=head, rows=d_rows)
        for i, o in enumerate(Os):
            got = _get(ys[i], (M, o), act if outs[i] == orn.OUT_ACT else 0)
            y = h @ W[i].T.astype(np.float64) + (base if outs[i] == orn.OUT_ADD else 0)
            # (a prologue's row may round to the other of two bf16 neighbours)
            _close(got, y, act, (pre, i), slack=4.0 if act == 0 else 1.0)
        for y in ys:
            y.free()
        if pre != orn.PRE_HEADS:
            g, u = (orn.Linear.dense(ctx, util.f32_to_bf16(_bf(rng.standard_normal((70,
                    K)) * K ** -0.5))) for _ in range(2))
            gw, uw = (util.bf16_to_f32(l.keep[0].download(np.uint16, (70, K))).astype(np.float64) for l in (g, u))
            y = ctx.alloc(M * 70 * 4)
            orn.dense_rows(ctx, adt, d_xa if pre == orn.PRE_NONE else d_x, M, K, [g, u], [y, None], [0, 0], pre=pre,
                    norm_w=d_wn,
                           w_offset=1.0, eps=1e-5, pair_act=orn.PAIR_GELU, rows=d_rows)
            _close(_get(y, (M, 70), act), R.gelu_tanh(h @ gw.T) * (h @ uw.T), act, ("gelu pair", pre),
                    slack=6.0 if act == 0 else 1.5)
            for b in (y, g, u):
                b.free()
    for b in [d_x, d_g, d_wn, d_xa, d_rows] + lins:
        b.free()


def test_dense_rows_of_a_call_are_those_of_single_rows(orn, ctx):
    """Below the GEMM widths a row of a call has the bits of the row alone."""
    rng = np.random.default_rng(5)
    M, K = 7, 640
    x = rng.standard_normal((M, K)).astype(np.float32)
    lin = orn.Linear.dense(ctx, util.f32_to_bf16(rng.standard_normal((48, K)).astype(np.float32)))
    wn = ctx.to_device(util.f32_to_bf16(0.1 * rng.standard_normal(K).astype(np.float32)))

    def run(rows):
        d, y = ctx.to_device(rows), ctx.alloc(len(rows) * 48 * 4)
        orn.dense_rows(ctx, orn.BF16, d, len(rows), K, [lin], [y], [orn.OUT_F32], pre=orn.PRE_NORM, norm_w=wn, w_offset=1.0)
        out = y.download(np.float32, (len(rows), 48))
        d.free()
        y.free()
        return out

    whole = run(x)
    assert np.array_equal(whole, np.concatenate([run(x[i:i + 1]) for i in range(M)]))
    lin.free()
    wn.free()


@pytest.mark.parametrize("act", [0, 1])
@pytest.mark.parametrize("heads,head", [(1, 64), (5, 24), (3, 17), (4, 512)])
def test_rows_of_the_prologues_alone(orn, ctx, act, heads, head):
    rng = np.random.default_rng(heads * 1000 + head)
    T, n = 9, heads * head
    x, gate, w = rng.standard_normal((T, n)).astype(np.float32), _bf(rng.standard_normal((T,
            n))), _bf(rng.standard_normal(n))
    d, g, dw, out = ctx.to_device(x), _dev(ctx, gate, act), ctx.to_device(util.f32_to_bf16(w)), ctx.alloc(T * n * 4)
    adt = orn.F32 if act == 0 else orn.BF16
    orn.norm_rows(ctx, d, dw, 1.0, T, n, 1e-4, adt, out)
    _close(_get(out, (T, n), act), R.norm_zero_centred(x.astype(np.float64), w, 1e-4), act, "norm")
    orn.head_norm_gate(ctx, d, dw, g, T, heads, head, 1e-4, adt, out)
    _close(_get(out, (T, n), act), R.rms(x.astype(np.float64).reshape(T, heads, head), 1e-4).reshape(T,
            n) * w * R.sigmoid(gate.astype(np.float64)),
           act, "head norm")
    for b in (d, g, dw, out):
        b.free()


# ---- mLSTM ------------------------------------------------------------------------------------
class Memory:
    """One mLSTM layer's memory on the device and in the reference."""

    def __init__(self, orn, ctx, H, dim, vdim, cap, act, slots=2, seed=0, f_bias=1.0):
        rng = np.random.default_rng(seed)
        self.orn, self.ctx, self.H, self.dim, self.vdim, self.cap, self.act = orn, ctx, H, dim, vdim, cap, act
        self.bi, self.bf = _bf(rng.standard_normal(H)), _bf(rng.standard_normal(H) + f_bias)
        self.d_b = [ctx.to_device(util.f32_to_bf16(b)) for b in (self.bi, self.bf)]
        self.floats, self.n, self.cur = orn.mlstm_state_floats(H, dim, vdim), slots, 0
        self.slots = ctx.alloc(self.floats * slots * 4).zero()
        self.ref = [(np.zeros((dim, vdim)), np.zeros(dim), 0.0) for _ in range(H)]

    def inputs(self, rng, T):
        f = (lambda a: _bf(a)) if self.act else (lambda a: a.astype(np.float32))
        return dict(q=f(rng.standard_normal((T, self.H, self.dim))), k=f(rng.standard_normal((T, self.H, self.dim))),
                    v=f(rng.standard_normal((T, self.H, self.vdim))), gi=(2 * rng.standard_normal((T,
                            self.H))).astype(np.float32),
                    gf=(2 * rng.standard_normal((T, self.H)) + 2).astype(np.float32))

    def step(self, x, snapshots=False):
        """The call's outputs [T, H, vdim]; the state moves to the next slot (or the last snapshot's)."""
        T = len(x["q"])
        d = {n: (_dev(self.ctx, x[n], self.act) if n in "qkv" else self.ctx.to_device(x[n])) for n in ("q", "k", "v",
                "gi", "gf")}
        o, first = self.ctx.alloc(T * self.H * self.vdim * 4), (self.cur + 1) % self.n
        self.orn.mlstm(self.ctx, act=self.act, bi=self.d_b[0], bf=self.d_b[1], gate_cap=self.cap, T=T, H=self.H,
                dim=self.dim,
                       vdim=self.vdim, state_in=self.slots.ptr.value + self.cur * self.floats * 4, slots=self.slots, n_slots=self.n,
                       first_slot=first, snapshots=int(snapshots), o=o, **d)
        self.cur = (first + T - 1) % self.n if snapshots else first
        out = o.download(np.float32, (T, self.H, self.vdim))
        for b in list(d.values()) + [o]:
            b.free()
        return out

    def want(self, x):
        out = np.empty((len(x["q"]), self.H, self.vdim))
        for h in range(self.H):
            li = R.soft_cap(x["gi"][:, h].astype(np.float64) + self.bi[h], self.cap)
            lf = R.log_sigmoid(R.soft_cap(x["gf"][:, h].astype(np.float64) + self.bf[h], self.cap))
            out[:, h], self.ref[h] = R.mlstm_cell(x["q"][:, h].astype(np.float64) * self.dim ** -0.5, x["k"][:,
                    h].astype(np.float64),
                                                  x["v"][:, h].astype(np.float64), li, lf, self.ref[h])
        return out

    def state(self, slot=None):
        """Per head (S [dim, vdim], n, m) of a slot."""
        ds = (self.dim + 3) // 4 * 4
        a = self.slots.download(np.float32, (self.n, self.H, self.floats // self.H))[self.cur if slot is None else slot]
        rows = a[:, :(self.vdim + 1) * ds].reshape(self.H, self.vdim + 1, ds)
        assert np.all(rows[:, :, self.dim:] == 0)
        return [(rows[h, :self.vdim, :self.dim].T, rows[h, self.vdim, :self.dim], a[h,
                (self.vdim + 1) * ds]) for h in range(self.H)]

    def check_state(self, what, tol):
        for h, (S, n, m) in enumerate(self.state()):
            Sr, nr, mr = self.ref[h]
            for a, b in ((S, Sr), (n, nr)):
                assert np.abs(a - b).max() <= tol * (np.abs(b).max() + 1e-6), (what, h, float(np.abs(a - b).max()))
            assert abs(m - mr) <= 2e-5 * (1 + abs(mr)), (what, h, m, mr)

    def close(self):
        for b in self.d_b + [self.slots]:
            b.free()


def _near(got, want, tol, what):
    """Relative to the size of the head's row (outputs of one head share their denominator)."""
    scale = np.sqrt(np.mean(want ** 2, axis=-1, keepdims=True)) + 1e-3 * np.sqrt(np.mean(want ** 2)) + 1e-12
    err = np.abs(got - want) / scale
    assert np.all(np.isfinite(got)) and err.max() <= tol, (what, float(err.max()), np.unravel_index(err.argmax(),
            err.shape))


@pytest.mark.parametrize("act", [0, 1])
@pytest.mark.parametrize("H,dim,vdim,cap", [(1, 16, 16, 5.0), (3, 10, 14, 4.0), (2, 72, 136, 9.0), (2, 136, 40, 15.0), (1,
        256, 192, 8.0),
                                            (2, 24, 300, 6.0), (1, 300, 20, 6.0)])
def test_mlstm_portions(orn, ctx, act, H, dim, vdim, cap):
    """Calls of many lengths one after the other, around the chunk's edges and the sixteen-column
    workgroups: outputs and state against the token-by-token reference. The outputs divide by
    max(|n . q|, e^-m), so an output is compared where that is not a difference of large numbers."""
    mem, rng = Memory(orn, ctx, H, dim, vdim, cap, act, seed=dim), np.random.default_rng(vdim)
    for T in (1, 3, 64, 2, 65, 63, 130, 1, 200, 8):
        x = mem.inputs(rng, T)
        got, want = mem.step(x), mem.want(x)
        _near(got, want, 2e-3 if act else 1e-3, (T, "outputs"))
        mem.check_state((T, "state"), 2e-4 if act else 2e-5)
    mem.close()


@pytest.mark.parametrize("act", [0, 1])
@pytest.mark.parametrize("far", [1, 63, 64, 127, 300])
def test_mlstm_finds_a_far_key(orn, ctx, act, far):
    """One token's input gate stands out and nothing is forgotten: `far` tokens later a query along its key
    must return its value, in a prompt and decoded alone; without that token it would not."""
    H, dim, vdim, at = 2, 40, 24, 5
    mem, rng = Memory(orn, ctx, H, dim, vdim, 12.0, act, seed=9, f_bias=9.0), np.random.default_rng(7)
    T = at + far + 1
    x = mem.inputs(rng, T)
    x["gf"][:] = 6.0
    x["gi"][:] = -6.0
    x["gi"][at] = 9.0
    x["q"][-1] = x["k"][at]
    for cut in (T, T - 1):
        m2 = Memory(orn, ctx, H, dim, vdim, 12.0, act, seed=9, f_bias=9.0)
        got = np.concatenate([m2.step({n: a[:cut] for n, a in x.items()})] + ([m2.step({n: a[cut:] for n,
                a in x.items()})] if cut < T else []))
        want = m2.want(x)
        _near(got[-1:], want[-1:], 2e-3, (far, cut))
        lost = {n: a.copy() for n, a in x.items()}
        lost["gi"][at] = -6.0
        m2.ref = [(np.zeros((dim, vdim)), np.zeros(dim), 0.0) for _ in range(H)]
        assert np.abs(m2.want(lost)[-1] - want[-1]).max() > 0.5
        m2.close()
    mem.close()


@pytest.mark.parametrize("act", [0, 1])
def test_mlstm_hard_gates(orn, ctx, act):
    """Gates at both of their ends: memory dropped and built up again from token to token, the running
    maximum far from zero on either side, denominators held up by e^-m alone."""
    mem, rng = Memory(orn, ctx, 2, 24, 16, 30.0, act, seed=2), np.random.default_rng(3)
    for T in (70, 5, 150):
        x = mem.inputs(rng, T)
        x["gi"] = (12 * rng.standard_normal((T, 2))).astype(np.float32)
        x["gf"] = (25 * rng.standard_normal((T, 2))).astype(np.float32)
        _near(mem.step(x), mem.want(x), 5e-3, T)
        mem.check_state(T, 3e-4)
    mem.close()


@pytest.mark.parametrize("act", [0, 1])
def test_mlstm_snapshots(orn, ctx, act):
    """With snapshots every token's state lands in its own slot of the ring; going on from slot keep - 1 is
    never having seen the rest."""
    mem, rng = Memory(orn, ctx, 2, 12, 20, 7.0, act, slots=5, seed=4), np.random.default_rng(5)
    x0, x1, x2 = mem.inputs(rng, 6), mem.inputs(rng, 4), mem.inputs(rng, 3)
    mem.step(x0)
    mem.want(x0)
    base = mem.cur
    mem.step(x1, snapshots=True)
    for keep in (1, 2, 3, 4):
        mem.cur = (base + keep) % 5
        saved = list(mem.ref)
        mem.want({n: a[:keep] for n, a in x1.items()})
        mem.check_state(keep, 2e-5)
        if keep < 4:
            mem.ref = saved
    _near(mem.step(x2), mem.want(x2), 2e-3 if act else 1e-3, "after")
    mem.close()


# ---- differential attention ---------------------------------------------------------------------
class Attention:
    """One attention layer's cache on the device and in the reference (ref: a diff_attention over raw rows)."""

    def __init__(self, orn, ctx, act, H, G, dim, vdim, size, keep, rot, base=1000.0, factor=1.0, scale=None, diff=0.45,
            lam=0.6, cap=700):
        self.orn, self.ctx, self.act = orn, ctx, act
        self.p = dict(H=H, G=G, dim=dim, vdim=vdim)
        self.size, self.keep, self.rot, self.base, self.factor = size, keep, rot, base, factor
        self.scale, self.diff, self.lam, self.cap, self.offset = dim ** -0.5 if scale is None else scale, diff, lam, cap, 0
        es = 4 if act == 0 else 2
        self.kc, self.vc = ctx.alloc(G * cap * 2 * dim * es), ctx.alloc(G * cap * vdim * es)
        # a used cache: nothing past the rows a call has written may be read
        for b in (self.kc, self.vc):
            b.upload(np.full(b.nbytes // 2, 0x7FC0, np.uint16))
        half = max(rot // 2, 1)
        ang = np.arange(cap)[:, None] * base ** (-2.0 * np.arange(half) / max(rot, 1)) / factor
        self.d_cos, self.d_sin = ctx.to_device(np.cos(ang).astype(np.float32)), ctx.to_device(np.sin(ang).astype(np.float32))
        self.K, self.V = [], []

    def inputs(self, rng, T, std=1.0):
        f = (lambda a: _bf(a)) if self.act else (lambda a: a.astype(np.float32))
        p = self.p
        return dict(q=f(std * rng.standard_normal((T, p["H"], 2, p["dim"]))), k=f(std * rng.standard_normal((T, p["G"], 2,
                p["dim"]))),
                    v=f(rng.standard_normal((T, p["G"], p["vdim"]))), gate=rng.standard_normal((T,
                            p["H"])).astype(np.float32))

    def step(self, x):
        T, p = len(x["q"]), self.p
        d = {n: (_dev(self.ctx, x[n], self.act) if n != "gate" else self.ctx.to_device(x[n])) for n in x}
        out, qr = self.ctx.alloc(T * p["H"] * p["vdim"] * 4), self.ctx.alloc(T * p["H"] * 2 * p["dim"] * 4)
        self.orn.diff_attn(self.ctx, act=self.act, cos=self.d_cos, sin=self.d_sin, rope_dims=self.rot,
                table_npos=self.cap, T=T,
                           offset=self.offset, cap=self.cap, window=self.size, keep_first=self.keep, scale=self.scale, lam=self.lam,
                           diff=self.diff, eps=1e-5, k_cache=self.kc, v_cache=self.vc, q_rot=qr, out=out, **d, **p)
        self.offset += T
        got = _get(out, (T, p["H"], p["vdim"]), self.act)
        for b in list(d.values()) + [out, qr]:
            b.free()
        return got

    def want(self, x, size=None, keep=None):
        p, size, keep = self.p, self.size if size is None else size, self.keep if keep is None else keep
        K, V, out = list(self.K), list(self.V), []
        for t in range(len(x["q"])):
            i = len(K)
            turn = lambda a: R.rope_interleaved(a.astype(np.float64), i, self.rot, self.base, self.factor)
            rnd = _bf if self.act else (lambda a: a)
            K.append(rnd(turn(x["k"][t])).astype(np.float64))
            V.append(x["v"][t].astype(np.float64))
            q, Ka, Va, row = rnd(turn(x["q"][t])).astype(np.float64), np.array(K), np.array(V), []
            for h in range(p["H"]):
                g = h // (p["H"] // p["G"])
                a1, a2 = (R.attend(q[h, m], Ka[:, g, m], Va[:, g], i, self.scale, size, keep) for m in (0, 1))
                row.append(R.rms(a1 - self.lam * a2, 1e-5) * (1 - self.diff) * R.sigmoid(float(x["gate"][t, h])))
            out.append(row)
        if size == self.size and keep == self.keep:
            self.K, self.V = K, V
        return np.array(out)

    def close(self):
        for b in (self.kc, self.vc, self.d_cos, self.d_sin):
            b.free()


SHAPES = [  # H, G, dim, vdim, size, keep, rot
    (2, 1, 16, 16, 5, 2, 8), (4, 4, 32, 64, 64, 0, 32), (6, 2, 24, 40, 65, 3, 4), (4, 1, 72, 136, 100, 70, 72),
    (2, 2, 128, 256, 33, 128, 64), (2, 1, 14, 9, 20, 7, 6), (3, 1, 6, 10, 1, 1, 2), (2, 1, 8, 8, 0, 0, 0), (4, 2, 64, 128,
            1000, 20, 32)]


@pytest.mark.parametrize("act", [0, 1])
@pytest.mark.parametrize("shape", SHAPES)
def test_attention_portions(orn, ctx, act, shape):
    """Portions of many lengths (decode and matrix-core widths) into one cache of garbage, windows shorter
    and longer than a key block, kept tokens fewer and more than a block, grouped heads."""
    H, G, dim, vdim, size, keep, rot = shape
    att, rng = Attention(orn, ctx, act, H, G, dim, vdim, size, keep, rot,
            factor=2.0), np.random.default_rng(dim * 31 + vdim)
    for T in (1, 2, 40, 1, 64, 33, 3, 100, 1, 7):
        x = att.inputs(rng, T)
        _close(att.step(x), att.want(x), act, (shape, T), slack=4.0 if act == 0 else 1.5)
    att.close()


@pytest.mark.parametrize("act", [0, 1])
@pytest.mark.parametrize("size,keep", [(64, 20), (72, 0), (5, 64), (130, 65), (1, 1)])
def test_attention_edges(orn, ctx, act, size, keep):
    """One key stands out for the first map and sits just inside, then just outside, the window or the kept
    first tokens: seen by a prompt's row and by a decoded one exactly where it should be. The reference
    with a window one longer or shorter, or one kept token more or fewer, is far away at these rows."""
    H, G, dim, vdim, rot = 2, 1, 24, 24, 8
    n = 230
    spots = sorted({j for j in (0, keep - 1, keep, keep + 1, 63, 64, n - 1 - size, n - size, n - size + 1,
            n - 2) if 0 <= j < n - 1})
    for spot in spots:
        rng = np.random.default_rng(spot)
        att = Attention(orn, ctx, act, H, G, dim, vdim, size, keep, rot)
        x = att.inputs(rng, n, std=0.2)
        u = _bf(np.where(np.arange(dim) >= rot, 2.5, 0.0))  # untouched by the rotation: distance does not matter
        x["q"][:, :, 0] = u
        x["k"][:, :, 0] = 0
        x["k"][spot, :, 0] = u
        want = att.want(x)
        seen = R.visible(n - 1, spot, size, keep)
        for cut in (n, n - 1):
            a2 = Attention(orn, ctx, act, H, G, dim, vdim, size, keep, rot)
            got = np.concatenate([a2.step({k: a[:cut] for k, a in x.items()})] + ([a2.step({k: a[cut:] for k,
                    a in x.items()})] if cut < n else []))
            _close(got[-3:], want[-3:], act, (spot, cut), slack=4.0 if act == 0 else 1.5)
            a2.close()
        for other in ((size + 1, keep), (max(size - 1, 1), keep), (size, keep + 1), (size, max(keep - 1, 0))):
            if R.visible(n - 1, spot, *other) != seen:
                fresh = Attention(orn, ctx, act, H, G, dim, vdim, size, keep, rot)
                assert np.abs(fresh.want(x, *other)[-1] - want[-1]).max() > 0.1, (spot, other)
                fresh.close()
        att.close()


def test_attention_of_single_rows_does_not_depend_on_the_call(orn, ctx):
    """A decode-width row has the same bits alone and among others of its call."""
    rng = np.random.default_rng(6)
    a, b = (Attention(orn, ctx, 1, 4, 2, 32, 48, 70, 5, 16) for _ in range(2))
    for T in (90, 6):
        x = a.inputs(rng, T)
        if T == 90:
            a.step(x)
            b.step(x)
        else:
            whole = a.step(x)
            one = np.concatenate([b.step({k: v[i:i + 1] for k, v in x.items()}) for i in range(T)])
            assert np.array_equal(whole, one)
    a.close()
    b.close()


def test_refusals(orn, ctx):
    """Calls the kernels cannot run come back as errors from the host."""
    b = ctx.alloc(1 << 16)
    ok = dict(act=1, q=b, k=b, v=b, gate=b, cos=b, sin=b, rope_dims=4, table_npos=64, T=1, H=2, G=1, dim=8, vdim=8,
            offset=0, cap=64,
              window=4, keep_first=0, scale=1.0, lam=0.5, diff=0.5, eps=1e-6, k_cache=b, v_cache=b, q_rot=b, out=b)
    for bad in (dict(H=3, G=2), dict(rope_dims=3), dict(rope_dims=10), dict(offset=64), dict(offset=60, T=5),
            dict(table_npos=0), dict(window=-1)):
        with pytest.raises(orn.OrnithError):
            orn.diff_attn(ctx, **dict(ok, **bad))
    s = orn.mlstm_state_floats(1, 8, 8) * 4
    ok = dict(act=1, q=b, k=b, v=b, gi=b, gf=b, bi=b, bf=b, gate_cap=4.0, T=1, H=1, dim=8, vdim=8, state_in=b, slots=b,
            n_slots=2,
              first_slot=1, snapshots=0, o=b)
    for bad in (dict(dim=513), dict(first_slot=2), dict(first_slot=0), dict(T=2, snapshots=1), dict(gate_cap=0.0)):
        with pytest.raises(orn.OrnithError):
            orn.mlstm(ctx, **dict(ok, **bad))
    assert s < 1 << 15
    b.free()
