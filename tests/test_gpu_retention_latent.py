"""GPU: retention, latent attention and what comes with them (YaRN tables, normed embeddings, silu pairs and
gates, scaled sums, capped logits), each alone, against float64 (tests/ref_stack.py)."""
import numpy as np
import pytest

import ref_stack as R
import util
from test_gpu_stack import _bf, _close, _dev, _get

pytestmark = pytest.mark.gpu


# ---- tails, prologues, tables --------------------------------------------------------------------
@pytest.mark.parametrize("act", [0, 1])
@pytest.mark.parametrize("M,K,head", [(1, 96, 24), (3, 90, 15), (4, 1040, 80), (33, 200, 8), (70, 264, 264)])
def test_dense_rows_forms(orn, ctx, act, M, K, head):
    """Heads normed without a weight under a silu gate, silu pairs, sums times a factor onto the stream, capped
    outputs, at decode and GEMM widths."""
    rng = np.random.default_rng(M * 1009 + K)
    Os = [33, 64, 18]
    W = [_bf(2 * rng.standard_normal((o, K)) * K ** -0.5) for o in Os]
    lins = [orn.Linear.dense(ctx, util.f32_to_bf16(w)) for w in W]
    x = rng.standard_normal((M, K)).astype(np.float32)
    g = _bf(rng.standard_normal((M, K))) if act else rng.standard_normal((M, K)).astype(np.float32)
    h = R.rms(x.astype(np.float64).reshape(M, -1, head), 1e-5).reshape(M, K) * R.silu(g.astype(np.float64))
    h = _bf(h).astype(np.float64) if act else h
    base = rng.standard_normal((M, Os[1])).astype(np.float32)
    adt = orn.F32 if act == 0 else orn.BF16
    d_x, d_g, d_rows, d_h = ctx.to_device(x), _dev(ctx, g, act), ctx.alloc(M * K * 4), _dev(ctx, h, act)
    h = _get(d_h, (M, K), act).astype(np.float64)
    ys = [ctx.alloc(M * o * 4) for o in Os]
    ys[1].upload(base)
    orn.dense_rows(ctx, adt, d_x, M, K, lins, ys, [orn.OUT_ACT, orn.OUT_ADD, orn.OUT_F32], pre=orn.PRE_HEADS, gate=d_g,
                   eps=1e-5, head_dim=head, rows=d_rows, gate_act=orn.GATE_SILU, add_scale=-0.75, soft_cap=1.5)
    slack = 4.0 if act == 0 else 1.2
    _close(_get(ys[0], (M, Os[0]), act), R.soft_cap(h @ W[0].T, 1.5), act, "capped act", slack)
    _close(ys[1].download(np.float32, (M, Os[1])), base - 0.75 * (h @ W[1].T), act, "added", slack)
    _close(ys[2].download(np.float32, (M, Os[2])), R.soft_cap(h @ W[2].T, 1.5), act, "capped f32", slack)
    pair = [orn.Linear.dense(ctx, util.f32_to_bf16(_bf(rng.standard_normal((40, K)) * K ** -0.5))) for _ in range(2)]
    gw, uw = (util.bf16_to_f32(l.keep[0].download(np.uint16, (40, K))).astype(np.float64) for l in pair)
    y = ctx.alloc(M * 40 * 4)
    orn.dense_rows(ctx, adt, d_h, M, K, pair, [y, None], [0, 0], pair_act=orn.PAIR_SILU)
    _close(_get(y, (M, 40), act), R.silu(h @ gw.T) * (h @ uw.T), act, "silu pair", 6.0 if act == 0 else 1.5)
    for b in [d_x, d_g, d_rows, d_h, y] + ys + lins + pair:
        b.free()


@pytest.mark.parametrize("act", [0, 1])
@pytest.mark.parametrize("M,K,O,ff", [(1, 96, (33, 8), 40), (2, 2048, (1500, 700, 4), 3000), (5, 264, (64,), 9), (3, 91, (17, 5), 12),
                                      (40, 128, (96, 24), 200)])
def test_two_calls_in_one_launch(orn, ctx, act, M, K, O, ff):
    """Projections behind one norm and a gated pair behind another over the same rows: the bits of two calls,
    whether the workgroups suffice for every group of rows or have to be shared out."""
    rng = np.random.default_rng(M + K)
    lin = lambda o: orn.Linear.dense(ctx, util.f32_to_bf16(rng.standard_normal((o, K)).astype(np.float32) * K ** -0.5))
    plain, pair = [lin(o) for o in O], [lin(ff) for _ in range(2)]
    x, wn = ctx.to_device(rng.standard_normal((M, K)).astype(np.float32)), [ctx.to_device(util.f32_to_bf16(
        1 + 0.3 * rng.standard_normal(K).astype(np.float32))) for _ in range(2)]
    rows, adt = ctx.alloc(M * K * 4), orn.F32 if act == 0 else orn.BF16
    got = []
    for one in (False, True):
        ys, up = [ctx.alloc(M * o * 4).zero() for o in O], ctx.alloc(M * ff * 4).zero()
        calls = [orn.dense_call(adt, x, M, K, plain, ys, [orn.OUT_F32] * len(O), pre=orn.PRE_NORM, norm_w=wn[0], rows=rows),
                 orn.dense_call(adt, x, M, K, pair, [up, None], [0, 0], pre=orn.PRE_NORM, norm_w=wn[1], pair_act=orn.PAIR_SILU,
                                rows=rows)]
        if one:
            orn.dense_rows_duo(ctx, calls)
        else:
            for c in calls:
                orn.dense_rows(ctx, c)
        got.append([y.download(np.float32, (M, o)) for y, o in zip(ys, O)] + [_get(up, (M, ff), act)])
        assert all(np.any(a) for a in got[-1])
        for b in ys + [up]:
            b.free()
    assert all(np.array_equal(a, b) for a, b in zip(*got))
    for b in plain + pair + wn + [x, rows]:
        b.free()


@pytest.mark.parametrize("n", [64, 91, 1000, 8200])
def test_embedded_rows_are_normed(orn, ctx, n):
    rng = np.random.default_rng(n)
    table, w = _bf(rng.standard_normal((17, n))), _bf(1 + 0.3 * rng.standard_normal(n))
    lin, d_w = orn.Linear.dense(ctx, util.f32_to_bf16(table)), ctx.to_device(util.f32_to_bf16(w))
    ids = np.array([3, 16, 0, 3, 9], np.uint32)
    d_ids, out = ctx.to_device(ids), ctx.alloc(5 * n * 4)
    for off in (0.0, 1.0):
        orn.embed_norm_rows(ctx, lin, d_ids, 5, d_w, off, 1e-3, out)
        want = R.rms(table[ids].astype(np.float64), 1e-3) * (off + w)
        _close(out.download(np.float32, (5, n)), want, 0, off)
    for b in (lin, d_w, d_ids, out):
        b.free()


@pytest.mark.parametrize("dims,base,sc", [(32, 1e4, dict(factor=8.0, original=2048, fast=32.0, slow=1.0)),
                                          (6, 50.0, dict(factor=1.0, original=64, fast=8.0, slow=1.0)),
                                          (64, 1e6, dict(factor=2.5, original=300, fast=500.0, slow=0.5)),
                                          (8, 20.0, dict(factor=4.0, original=4000, fast=2.0, slow=1.9))])
def test_yarn_tables(orn, ctx, dims, base, sc):
    """Ramps inside the pairs, before the first, past the last, and of no length."""
    n, half = 700, dims // 2
    c, s = ctx.alloc(n * half * 4), ctx.alloc(n * half * 4)
    orn.rope_table_yarn(ctx, n, dims, base, sc["factor"], sc["original"], sc["fast"], sc["slow"], c, s)
    f, gain = R.turn_frequencies(dims, base, sc)
    a = np.arange(n)[:, None] * f
    for buf, want in ((c, np.cos(a)), (s, np.sin(a))):
        assert np.abs(buf.download(np.float32, (n, half)) - gain * want).max() < 1e-6 * gain
        buf.free()


# ---- retention -------------------------------------------------------------------------------------
class State:
    """One retention layer's state on the device and in the reference."""

    def __init__(self, orn, ctx, H, dim, vdim, decay, rot, act, slots=2, cap=1200, base=300.0):
        self.orn, self.ctx, self.H, self.dim, self.vdim, self.act, self.decay = orn, ctx, H, dim, vdim, act, decay
        self.floats, self.n, self.cur, self.at, self.rot, self.cap = orn.retention_state_floats(H, dim, vdim), slots, 0, 0, rot, cap
        self.slots = ctx.alloc(self.floats * slots * 4).zero()
        self.pw = ctx.alloc(H * orn.DECAY_POWERS * 4)
        orn.decay_powers(ctx, decay, self.pw)
        self.freqs, _ = R.turn_frequencies(rot, base) if rot else (np.zeros(0), 1)
        a = np.arange(cap)[:, None] * (self.freqs if rot else np.zeros(1))
        self.d_cos, self.d_sin = ctx.to_device(np.cos(a).astype(np.float32)), ctx.to_device(np.sin(a).astype(np.float32))
        self.ref = [np.zeros((dim, vdim)) for _ in range(H)]
        self.ref_at = 0

    def inputs(self, rng, T):
        f = (lambda a: _bf(a)) if self.act else (lambda a: a.astype(np.float32))
        return {n: f(rng.standard_normal((T, self.H, d))) for n, d in (("q", self.dim), ("k", self.dim), ("v", self.vdim))}

    def step(self, x, snapshots=False):
        T = len(x["q"])
        d = {n: _dev(self.ctx, x[n], self.act) for n in x}
        o, first = self.ctx.alloc(T * self.H * self.vdim * 4), (self.cur + 1) % self.n
        self.orn.retention(self.ctx, act=self.act, cos=self.d_cos, sin=self.d_sin, rope_dims=self.rot, table_npos=self.cap,
                           offset=self.at, decay=self.pw, T=T, H=self.H, dim=self.dim, vdim=self.vdim,
                           state_in=self.slots.ptr.value + self.cur * self.floats * 4, slots=self.slots, n_slots=self.n,
                           first_slot=first, snapshots=int(snapshots), o=o, **d)
        self.cur = (first + T - 1) % self.n if snapshots else first
        self.at += T
        out = o.download(np.float32, (T, self.H, self.vdim))
        for b in list(d.values()) + [o]:
            b.free()
        return out

    def want(self, x):
        T, out = len(x["q"]), np.empty((len(x["q"]), self.H, self.vdim))
        q, k = (np.array([R.turn(x[n][t].astype(np.float64), self.ref_at + t, self.freqs, 1.0, True) for t in range(T)]) for n in "qk")
        for h in range(self.H):
            out[:, h], self.ref[h] = R.retention_cell(q[:, h], k[:, h] * self.dim ** -0.5, x["v"][:, h].astype(np.float64),
                                                      self.decay[h], self.ref[h])
        self.ref_at += T
        return out

    def check_state(self, what, tol):
        ds = (self.dim + 3) // 4 * 4
        a = self.slots.download(np.float32, (self.n, self.H, self.vdim, ds))[self.cur]
        assert np.all(a[:, :, self.dim:] == 0)
        for h in range(self.H):
            err = np.abs(a[h, :, :self.dim].T - self.ref[h]).max()
            assert err <= tol * (np.abs(self.ref[h]).max() + 1e-6), (what, h, float(err))

    def close(self):
        for b in (self.slots, self.pw, self.d_cos, self.d_sin):
            b.free()


def _near(got, want, tol, what):
    """Relative to the size of the outputs of the head."""
    scale = np.sqrt(np.mean(want ** 2, axis=(0, 2), keepdims=True)) + 1e-12
    err = np.abs(got - want) / scale
    assert np.all(np.isfinite(got)) and err.max() <= tol, (what, float(err.max()), np.unravel_index(err.argmax(), err.shape))


DECAYS = (0.999, 0.5, 1.0, 0.0, -0.75)


@pytest.mark.parametrize("act", [0, 1])
@pytest.mark.parametrize("H,dim,vdim,rot", [(1, 16, 16, 16), (3, 10, 14, 6), (2, 72, 136, 40), (5, 136, 40, 136), (1, 256, 192, 4),
                                            (2, 24, 300, 0), (1, 300, 20, 300), (4, 64, 64, 12)])
def test_retention_portions(orn, ctx, act, H, dim, vdim, rot):
    """Calls of many lengths one after the other, around the chunk's edges and the sixteen-column workgroups:
    outputs and state against the token-by-token reference."""
    st, rng = State(orn, ctx, H, dim, vdim, [DECAYS[(h + dim) % 5] for h in range(H)], rot, act), np.random.default_rng(vdim)
    for T in (1, 3, 64, 2, 65, 63, 130, 1, 200, 8):
        x = st.inputs(rng, T)
        _near(st.step(x), st.want(x), 1e-4 if act else 2e-5, (T, "outputs"))
        st.check_state((T, "state"), 1e-4 if act else 1e-5)
    st.close()


@pytest.mark.parametrize("act", [0, 1])
@pytest.mark.parametrize("far", [1, 63, 64, 127, 700])
def test_retention_finds_a_far_key(orn, ctx, act, far):
    """One key stands out: `far` tokens later a query along it must return its value, faded by the head's
    decay, in a prompt and decoded alone; without that token it would not."""
    H, dim, vdim, at, rot = 2, 40, 24, 5, 8
    decay, rng, T = (1.0, 0.998), np.random.default_rng(7), at + far + 1
    st = State(orn, ctx, H, dim, vdim, decay, rot, act)
    x = st.inputs(rng, T)
    x["k"] = _bf(0.05 * x["k"])
    u = np.where(np.arange(dim) >= rot, 2.0, 0.0)  # untouched by the rotation: distance does not matter
    x["k"][at] = u
    x["q"][-1] = u
    for cut in (T, T - 1):
        s2 = State(orn, ctx, H, dim, vdim, decay, rot, act)
        got = np.concatenate([s2.step({n: a[:cut] for n, a in x.items()})] + ([s2.step({n: a[cut:] for n,
                a in x.items()})] if cut < T else []))
        want = s2.want(x)
        assert np.abs(got[-1] - want[-1]).max() <= 2e-4 * np.abs(want[-1]).max(), (far, cut)
        lost = {n: a.copy() for n, a in x.items()}
        lost["k"][at] = 0
        s2.ref, s2.ref_at = [np.zeros((dim, vdim)) for _ in range(H)], 0
        assert np.abs(s2.want(lost)[-1] - want[-1]).max() > 0.3 * np.abs(want[-1]).max()
        s2.close()
    st.close()


@pytest.mark.parametrize("act", [0, 1])
def test_retention_snapshots(orn, ctx, act):
    """With snapshots every token's state lands in its own slot of the ring; going on from slot keep - 1 is
    never having seen the rest."""
    st, rng = State(orn, ctx, 2, 12, 20, (0.9, 1.0), 6, act, slots=5), np.random.default_rng(5)
    x0, x1, x2 = st.inputs(rng, 6), st.inputs(rng, 4), st.inputs(rng, 3)
    st.step(x0)
    st.want(x0)
    base = st.cur
    st.step(x1, snapshots=True)
    for keep in (1, 2, 3, 4):
        st.cur = (base + keep) % 5
        saved, at = list(st.ref), st.ref_at
        st.want({n: a[:keep] for n, a in x1.items()})
        st.check_state(keep, 1e-5)
        if keep < 4:
            st.ref, st.ref_at = saved, at
    _near(st.step(x2), st.want(x2), 2e-5, "after")
    st.close()


# ---- latent attention --------------------------------------------------------------------------------
class Latent:
    """One latent-attention layer and its cache on the device and in the reference. `of`: another layer's
    Latent whose rows this one reads."""

    def __init__(self, orn, ctx, act, H, dim, rot, vdim, rank, size, scale=None, sink=True, gate=True, seed=0, cap=700, of=None):
        rng = np.random.default_rng(seed)
        self.orn, self.ctx, self.act, self.of = orn, ctx, act, of
        self.p = dict(H=H, dim=dim, rot_dim=rot, vdim=vdim, rank=rank)
        self.size, self.cap, self.offset = size, cap, 0
        self.scale = (dim + rot) ** -0.5 if scale is None else scale
        self.uk, self.uv = _bf(1.5 * rng.standard_normal((H * dim, rank)) * rank ** -0.5), _bf(rng.standard_normal((H * vdim, rank)) * rank ** -0.5)
        self.norm, self.sink, self.gate = _bf(1 + 0.3 * rng.standard_normal(rank)), _bf(2 * rng.standard_normal(H)) if sink else None, gate
        self.lin = [orn.Linear.dense(ctx, util.f32_to_bf16(m)) for m in (self.uk, self.uv)]
        self.d_norm = ctx.to_device(util.f32_to_bf16(self.norm))
        self.d_sink = ctx.to_device(util.f32_to_bf16(self.sink)) if sink else None
        es = 4 if act == 0 else 2
        self.freqs, self.gain = R.turn_frequencies(rot, 500.0, dict(factor=3.0, original=100, fast=6.0, slow=1.0))
        a = np.arange(cap)[:, None] * self.freqs
        self.d_cos, self.d_sin = (ctx.to_device((self.gain * f(a)).astype(np.float32)) for f in (np.cos, np.sin))
        self.own = []
        if of is None:
            self.cc, self.rc, self.C, self.K = ctx.alloc(cap * rank * es), ctx.alloc(cap * rot * es), [], []
            # a used cache: nothing past the rows a call has written may be read
            for b in (self.cc, self.rc):
                b.upload(np.full(b.nbytes // 2, 0x7FC0, np.uint16))
            self.own = [self.cc, self.rc]

    def inputs(self, rng, T):
        p, f = self.p, (lambda a: _bf(a)) if self.act else (lambda a: a.astype(np.float32))
        return dict(q=f(rng.standard_normal((T, p["H"], p["dim"] + p["rot_dim"]))),
                    down=rng.standard_normal((T, p["rank"] + p["rot_dim"])).astype(np.float32),
                    gate=rng.standard_normal((T, p["H"])).astype(np.float32))

    def step(self, x):
        T, p, src = len(x["q"]), self.p, self.of or self
        q, down, g = _dev(self.ctx, x["q"], self.act), self.ctx.to_device(x["down"]), self.ctx.to_device(x["gate"])
        out = self.ctx.alloc(T * p["H"] * p["vdim"] * 4)
        self.orn.latent_attn(self.ctx, act=self.act, q=q, down=down if self.of is None else None, down_norm=self.d_norm,
                             uk=self.lin[0], uv=self.lin[1], gate=g if self.gate else None, sink=self.d_sink, cos=self.d_cos,
                             sin=self.d_sin, table_npos=self.cap, T=T, offset=self.offset, cap=self.cap, window=self.size,
                             scale=self.scale, eps=1e-5, c_cache=src.cc, r_cache=src.rc, out=out, **p)
        self.offset += T
        got = _get(out, (T, p["H"], p["vdim"]), self.act)
        for b in (q, down, g, out):
            b.free()
        return got

    def want(self, x, size=None, sink=True, commit=True, rows=None):
        """rows: only the call's last ones are worked out (the others come back as zeros)."""
        p, rnd = self.p, _bf if self.act else (lambda a: a)
        H, d, dv, rank = p["H"], p["dim"], p["vdim"], p["rank"]
        src, size = self.of or self, self.size if size is None else size
        C, K, out, T = list(src.C), list(src.K), [], len(x["q"])
        at = len(C) - (T if self.of else 0)
        for t in range(T):
            i, dn = at + t, x["down"][t].astype(np.float64)
            if self.of is None:
                C.append(rnd(R.norm_plain(dn[:rank], self.norm, 1e-5)).astype(np.float64))
                K.append(rnd(R.turn(dn[rank:], i, self.freqs, self.gain, False)).astype(np.float64))
            if rows is not None and t < T - rows:
                out.append(np.zeros((H, dv)))
                continue
            js = [j for j in range(i + 1) if R.visible(i, j, size, 0)]
            c, kr, row = np.array([C[j] for j in js]), np.array([K[j] for j in js]), []
            for h in range(H):
                q = x["q"][t, h].astype(np.float64)
                s = ((c @ self.uk[h * d:(h + 1) * d].T) @ q[:d] + kr @ R.turn(q[d:], i, self.freqs, self.gain, False)) * self.scale
                o = R.attend_sink(s, c @ self.uv[h * dv:(h + 1) * dv].T, float(self.sink[h]) if self.d_sink and sink else -1e30)
                row.append(o * (R.sigmoid(float(x["gate"][t, h])) if self.gate else 1.0))
            out.append(row)
        if commit and self.of is None:
            self.C, self.K = C, K
        return np.array(out)

    def close(self):
        for b in self.own + self.lin + [self.d_norm, self.d_cos, self.d_sin] + ([self.d_sink] if self.d_sink else []):
            b.free()


SHAPES = [  # H, dim, rot, vdim, rank, window
    (20, 16, 8, 16, 24, 5), (35, 8, 8, 8, 256, 90), (17, 24, 64, 40, 512, 50), (2, 16, 8, 16, 24, 5), (4, 32, 32, 64, 64, 64), (6, 24, 8, 40, 40, 65), (3, 72, 24, 136, 104, 100), (2, 128, 64, 256, 192, 33),
    (3, 14, 6, 9, 23, 20), (1, 7, 2, 3, 5, 1), (5, 40, 16, 48, 520, 0), (2, 192, 64, 128, 136, 1000), (7, 8, 8, 8, 8, 130)]


@pytest.mark.parametrize("act", [0, 1])
@pytest.mark.parametrize("shape", SHAPES)
def test_latent_portions(orn, ctx, act, shape):
    """Portions of many lengths (decode and matrix-core widths) into one cache of garbage, windows shorter and
    longer than a key block, one head and many, ranks past a wavefront's reach; without a sink and a gate too.
    In bf16 a prompt's keys and values are rounded where decoding has none, hence the slack."""
    la = Latent(orn, ctx, act, *shape, scale=-0.2 if shape[0] == 6 else None, sink=shape[0] != 7, gate=shape[0] != 7, seed=shape[1])
    rng = np.random.default_rng(shape[3])
    for T in (1, 2, 40, 1, 64, 33, 3, 100, 1, 7):
        x = la.inputs(rng, T)
        _close(la.step(x), la.want(x), act, (shape, T), slack=6.0 if act == 0 else 3.0)
    la.close()


@pytest.mark.parametrize("shape", [(18, 16, 8, 24, 320, 0), (3, 24, 8, 16, 40, 2300), (2, 16, 16, 24, 544, 2050)])
def test_latent_far_rows(orn, ctx, shape):
    """Thousands of rows in sight, where a decoded row's blocks grow longer; one early row stands out."""
    H, dim, rot, vdim, rank, size = shape
    la, rng, n = Latent(orn, ctx, 1, *shape, cap=3000), np.random.default_rng(rank), 2600
    x = la.inputs(rng, n)
    spot = n - 2000
    c = R.norm_plain(x["down"][spot, :rank].astype(np.float64), la.norm, 1e-5)
    tail = la.inputs(rng, 4)
    for q in (x["q"][-1], tail["q"][0], tail["q"][3]):
        for h in range(H):
            key = la.uk[dim * h:dim * h + dim] @ c
            q[h, :dim] = _bf(key * 12.0 / (key @ key) / la.scale)
    _close(la.step(x)[-3:], la.want(x, rows=3)[-3:], 1, "prompt", slack=3.0)
    for part in ({k: a[:1] for k, a in tail.items()}, {k: a[1:] for k, a in tail.items()}):
        _close(la.step(part), la.want(part), 1, "decoded", slack=3.0)
    la.close()


@pytest.mark.parametrize("act", [0, 1])
@pytest.mark.parametrize("size", [64, 72, 5, 130, 1])
def test_latent_window_edges(orn, ctx, act, size):
    """One row stands out for the last query and sits just inside, then just outside, the window, and at key
    blocks' edges: seen by a prompt's row and by a decoded one exactly where it should be. The reference with
    a window one longer or shorter is far away there."""
    shape, n = (2, 24, 8, 24, 32), 230
    for spot in sorted({j for j in (0, 63, 64, n - 1 - size, n - size, n - size + 1, n - 2, n - 33) if 0 <= j < n - 1}):
        rng = np.random.default_rng(spot)
        la = Latent(orn, ctx, act, *shape, size)
        x = la.inputs(rng, n)
        c = R.norm_plain(x["down"][spot, :32].astype(np.float64), la.norm, 1e-5)
        for h in range(2):
            key = la.uk[24 * h:24 * h + 24] @ c
            x["q"][-1, h] = 0
            x["q"][-1, h, :24] = _bf(key * 14.0 / (key @ key) / la.scale)
        want = la.want(x, commit=False)
        seen = R.visible(n - 1, spot, size, 0)
        for cut in (n, n - 1):
            b = Latent(orn, ctx, act, *shape, size)
            got = np.concatenate([b.step({k: a[:cut] for k, a in x.items()})] + ([b.step({k: a[cut:] for k,
                    a in x.items()})] if cut < n else []))
            _close(got[-3:], want[-3:], act, (spot, cut), slack=8.0 if act == 0 else 3.0)
            b.close()
        for other in (size + 1, max(size - 1, 1)):
            if R.visible(n - 1, spot, other, 0) != seen:
                assert np.abs(la.want(x, size=other, commit=False)[-1] - want[-1]).max() > 0.1, (spot, other)
        la.close()


@pytest.mark.parametrize("act", [0, 1])
def test_latent_sink_counts_once(orn, ctx, act):
    """A sink as large as the scores takes its share of every row, from the first token on; sinks far above
    and far below the scores leave nothing and everything."""
    la, rng = Latent(orn, ctx, act, 4, 24, 8, 24, 32, 40), np.random.default_rng(3)
    la.sink[:] = (3.0, 0.0, -40.0, 60.0)
    la.d_sink.upload(util.f32_to_bf16(la.sink))
    for T in (1, 50, 2, 60, 1):
        x = la.inputs(rng, T)
        without = la.want(x, sink=False, commit=False)
        got, want = la.step(x), la.want(x)
        _close(got, want, act, T, slack=6.0 if act == 0 else 3.0)
        assert np.abs(without[:, :2] - want[:, :2]).max() > 0.05 and np.abs(want[:, 3]).max() < 1e-9
        assert np.abs(without[:, 2] - want[:, 2]).max() < 1e-9
    la.close()


@pytest.mark.parametrize("act", [0, 1])
def test_latent_rows_of_another_layer(orn, ctx, act):
    """A layer without rows of its own reads the other's, through its own maps, heads and window."""
    a = Latent(orn, ctx, act, 3, 24, 16, 40, 48, 9, seed=1)
    b = Latent(orn, ctx, act, 5, 40, 16, 24, 48, 70, seed=2, of=a)
    rng = np.random.default_rng(4)
    for T in (1, 40, 2, 90, 1, 5):
        xa, xb = a.inputs(rng, T), b.inputs(rng, T)
        _close(a.step(xa), a.want(xa), act, ("own", T), slack=6.0 if act == 0 else 3.0)
        _close(b.step(xb), b.want(xb), act, ("other's", T), slack=6.0 if act == 0 else 3.0)
    a.close()
    b.close()


def test_latent_single_rows_do_not_depend_on_the_call(orn, ctx):
    """A decode-width row has the same bits alone and among others of its call."""
    rng = np.random.default_rng(6)
    a, b = (Latent(orn, ctx, 1, 4, 32, 16, 48, 72, 70) for _ in range(2))
    x = a.inputs(rng, 90)
    a.step(x)
    b.step(x)
    x = a.inputs(rng, 7)
    whole = a.step(x)
    assert np.array_equal(whole, np.concatenate([b.step({k: v[i:i + 1] for k, v in x.items()}) for i in range(7)]))
    a.close()
    b.close()


def test_retention_single_rows_do_not_depend_on_the_call(orn, ctx):
    rng = np.random.default_rng(8)
    a, b = (State(orn, ctx, 3, 40, 24, (0.9, 0.99, 1.0), 16, 1) for _ in range(2))
    x = a.inputs(rng, 30)
    whole = a.step(x)
    assert np.array_equal(whole, np.concatenate([b.step({k: v[i:i + 1] for k, v in x.items()}) for i in range(30)]))
    a.close()
    b.close()


def test_refusals(orn, ctx):
    """Calls the kernels cannot run come back as errors from the host."""
    b = ctx.alloc(1 << 16)
    lin = [orn.Linear.dense(ctx, np.zeros((16, 8), np.uint16)) for _ in range(2)]
    ok = dict(act=1, q=b, down=b, down_norm=b, uk=lin[0], uv=lin[1], gate=b, sink=b, cos=b, sin=b, table_npos=64, T=1, H=2, dim=8,
              rot_dim=4, vdim=8, rank=8, offset=0, cap=64, window=4, scale=1.0, eps=1e-6, c_cache=b, r_cache=b, out=b)
    for bad in (dict(H=3), dict(rot_dim=3), dict(offset=64), dict(offset=60, T=5), dict(table_npos=0), dict(window=-1), dict(rank=9),
                dict(down_norm=None), dict(cos=None)):
        with pytest.raises(orn.OrnithError):
            orn.latent_attn(ctx, **dict(ok, **bad))
    ok = dict(act=1, q=b, k=b, v=b, cos=b, sin=b, rope_dims=4, table_npos=64, offset=0, decay=b, T=1, H=1, dim=8, vdim=8, state_in=b,
              slots=b, n_slots=2, first_slot=1, snapshots=0, o=b)
    for bad in (dict(dim=513), dict(first_slot=2), dict(first_slot=0), dict(T=2, snapshots=1), dict(rope_dims=10), dict(rope_dims=5),
                dict(offset=64), dict(decay=None)):
        with pytest.raises(orn.OrnithError):
            orn.retention(ctx, **dict(ok, **bad))
    for x in [b] + lin:
        x.free()
