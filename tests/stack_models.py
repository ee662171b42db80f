"""Small layer-list models for the tests: configurations of odd and even sizes, random weights."""
import numpy as np

import util


def mlstm(heads, dim, vdim, cap, ff=None):
    return {"type": "mlstm", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "gate_cap": cap},
            "mlp": {"kind": "dense", "ff": ff} if ff else None}


def attention(heads, kv, dim, vdim, size, keep, rot=8, base=1000.0, factor=1.0, diff=0.4, ff=None, scale=None):
    return {"type": "attention", "mixer": {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "diff": diff,
                                           "scale": scale or dim ** -0.5, "mask": {"size": size, "keep_first": keep},
                                           "rot": {"base": base, "dims": rot, "scaling": {"factor": factor}}},
            "mlp": {"kind": "dense", "ff": ff} if ff else None}


def retention(heads, dim, vdim, decay, rot, base=1000.0, ff=None):
    return {"type": "retention", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "decay": list(decay),
                                           "rot": {"base": base, "dims": rot}},
            "mlp": {"kind": "dense", "ff": ff} if ff else None}


YARN = {"factor": 4.0, "original": 64, "fast": 8.0, "slow": 1.0}


def latent(heads, dim, rot_dim, vdim, rank, size, base=1000.0, scaling=None, kv_from=None, scale=None, ff=None):
    mx = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": rank,
          "scale": scale or (dim + rot_dim) ** -0.5, "rot": {"base": base, "dims": rot_dim}}
    if size:
        mx["mask"] = {"size": size}
    if scaling:
        mx["rot"]["scaling"] = scaling
    if kv_from is not None:
        mx["kv_from"] = kv_from
    return {"type": "latent_attention", "mixer": mx, "mlp": {"kind": "dense", "ff": ff} if ff else None}


def side_by_side(vocab, width, layers, mult, cap, eps=1e-5):
    return {"architecture": "Ranavik", "vocab": vocab, "width": width, "norm": {"eps": eps}, "residual_mult": mult,
            "logit_softcap": cap, "layers": layers}


def model(vocab, width, layers, eps=1e-5, scale=1.0):
    return {"architecture": "Pigodra", "vocab": vocab, "width": width, "norm": {"eps": eps}, "embedding": {"scale": scale},
            "layers": layers}


CONFIGS = {
    # every mixer with and without a feed-forward, all sizes multiples of 8, one KV head, window < block
    "even": model(320, 128, [attention(3, 1, 24, 40, 9, 3, rot=24, factor=3.0, ff=96), mlstm(2, 40, 24, 6.0, ff=160),
                             mlstm(1, 16, 72, 15.0), attention(4, 4, 16, 16, 33, 1, rot=2)], eps=1e-5, scale=2.0),
    # sizes that fit no vector load, grouped heads, kept tokens more than a block, no kept tokens
    "odd": model(211, 90, [mlstm(3, 10, 14, 4.0), attention(6, 2, 14, 9, 21, 70, rot=6, base=50.0, diff=0.7, ff=33),
                           attention(2, 1, 6, 10, 64, 0, rot=0, scale=-0.3), mlstm(5, 7, 3, 8.0, ff=19)], eps=1e-4, scale=0.25),
    # one kind of layer alone
    "memory": model(256, 64, [mlstm(2, 72, 136, 9.0, ff=64), mlstm(4, 24, 8, 12.0)]),
    "attention": model(256, 64, [attention(4, 2, 72, 136, 70, 5, rot=40, factor=1.5), attention(2, 2, 32, 64, 128, 64, rot=32, ff=72)]),
    # both mixers with and without a feed-forward, multiples of 8; a layer that reads another's rows through
    # a window of its own, with other heads
    "rv_even": side_by_side(320, 128, [latent(3, 24, 16, 40, 48, 9, scaling=YARN, ff=96), retention(2, 40, 24, (0.5, 0.97), 40, ff=160),
                                       latent(5, 56, 16, 16, 48, 33, scaling=YARN, kv_from=0), retention(1, 16, 72, (1.0,), 8)],
                            0.6, 7.0),
    # sizes that fit no vector load, decays from none to whole, a negative scale, no window, one head
    "rv_odd": side_by_side(211, 90, [retention(3, 10, 14, (0.0, 0.875, 0.999), 6, base=50.0, ff=33),
                                     latent(5, 14, 6, 9, 22, 21, base=200.0, scaling=dict(YARN, factor=1.0), scale=-0.3),
                                     latent(1, 7, 6, 10, 22, 0, base=200.0, scaling=dict(YARN, factor=1.0), kv_from=1, ff=19),
                                     retention(5, 6, 3, (0.25, 0.9, 0.75, 1.0, 0.96), 2)], 1.0, 40.0, eps=1e-4),
    # one kind of layer alone
    "rv_state": side_by_side(256, 64, [retention(2, 72, 136, (0.99, 0.998), 72, ff=64), retention(4, 24, 8, (0.5, 0.6, 0.7, 1.0), 0)],
                             0.8, 12.0),
    "rv_latent": side_by_side(256, 64, [latent(4, 72, 40, 136, 64, 70), latent(2, 32, 64, 64, 40, 128, base=5e4, scaling=YARN, ff=72),
                                        latent(2, 96, 64, 72, 40, 1, base=5e4, scaling=YARN, kv_from=1)], 1.25, 9.0),
}


def bf16(a):
    return util.bf16_to_f32(util.f32_to_bf16(np.asarray(a, np.float32)))


def weights(cfg, seed, gate_bias=2.0):
    """name -> float32 array of bf16 values. Scaled so that no mixer is drowned in the stream, gates reach
    both of their ends, and attention is far from uniform."""
    rng = np.random.default_rng(seed)
    W, V, out = cfg["width"], cfg["vocab"], {}

    def put(name, *shape, std=1.0, mean=0.0):
        out[name] = bf16(mean + std * rng.standard_normal(shape))

    put("embed", V, W)
    put("head", V, W, std=W ** -0.5)
    plain = 1.0 if cfg["architecture"] == "Ranavik" else 0.0  # norm weights as they are, or from one
    if plain:
        put("embed.norm", W, std=0.3, mean=1.0)
    put("final.norm", W, std=0.3, mean=plain)
    for i, layer in enumerate(cfg["layers"]):
        p, m, kind = f"l{i}.", layer["mixer"], layer["type"]
        put(p + "norm1", W, std=0.3, mean=plain)
        H = m["heads"]
        if kind == "mlstm":
            for n, o, s in (("q", H * m["dim"], 1.5), ("k", H * m["dim"], 1.5), ("v", H * m["vdim"], 1.0),
                            ("g", H * m["vdim"], 1.0), ("i", H, 2.0), ("f", H, 2.0)):
                put(p + "mix." + n, o, W, std=s * W ** -0.5)
            put(p + "mix.i.b", H, std=1.0, mean=-1.0)
            put(p + "mix.f.b", H, std=1.0, mean=gate_bias)
            put(p + "mix.norm", H * m["vdim"], std=0.3, mean=1.0)
        elif kind == "attention":
            G = m["kv_heads"]
            for n, o, s in (("q", H * 2 * m["dim"], 2.0), ("k", G * 2 * m["dim"], 2.0), ("v", G * m["vdim"], 1.0), ("g", H, 1.0)):
                put(p + "mix." + n, o, W, std=s * W ** -0.5)
            for n in ("lq1", "lk1", "lq2", "lk2"):
                put(p + "mix." + n, m["dim"], std=0.3)
        elif kind == "retention":
            for n, o in (("q", H * m["dim"]), ("k", H * m["dim"]), ("v", H * m["vdim"]), ("g", H * m["vdim"])):
                put(p + "mix." + n, o, W, std=1.5 * W ** -0.5)
        else:
            r, dr = m["kv_rank"], m["rot_dim"]
            put(p + "mix.q", H * (m["dim"] + dr), W, std=1.5 * W ** -0.5)
            put(p + "mix.g", H, W, std=W ** -0.5)
            if m.get("kv_from") is None:
                put(p + "mix.dkv", r + dr, W, std=1.5 * W ** -0.5)
                put(p + "mix.dkv.norm", r, std=0.3, mean=1.0)
            put(p + "mix.uk", H * m["dim"], r, std=1.5 * r ** -0.5)
            put(p + "mix.uv", H * m["vdim"], r, std=r ** -0.5)
            put(p + "mix.sink", H, std=1.5)
        put(p + "mix.o", W, H * m["vdim"], std=(H * m["vdim"]) ** -0.5)
        if layer["mlp"]:
            ff = layer["mlp"]["ff"]
            put(p + "norm2", W, std=0.3, mean=plain)
            put(p + "mlp.gate", ff, W, std=1.5 * W ** -0.5)
            put(p + "mlp.up", ff, W, std=W ** -0.5)
            put(p + "mlp.down", W, ff, std=ff ** -0.5)
    return out


def load(orn, ctx, cfg, w, act):
    """(store, model) on the device."""
    ws = orn.WeightStore(ctx)
    for n, a in w.items():
        ws.put(n, util.f32_to_bf16(a), orn.DT_BF16)
    return ws, orn.TextModel.from_json(ctx, ws, cfg, act)
