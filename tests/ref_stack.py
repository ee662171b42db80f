"""Plain float64 restatement of the layer-list designs (test infrastructure only): one function per
mechanism, written from its equations, token by token and head by head, sharing nothing with the
library. Weights are numpy arrays of any float type, keyed by the tensor names of the artifact.

A model here is (cfg, w): `cfg` the parsed config.json, `w` the name -> array map."""
import math

import numpy as np


def rms(x, eps):
    """x over its root mean square along the last axis, eps inside the root."""
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def norm_zero_centred(x, w, eps):
    """RMS norm whose weight is stored as its distance from one."""
    return rms(x, eps) * (1.0 + w)


def norm_plain(x, w, eps):
    """RMS norm with the weight as it is."""
    return rms(x, eps) * w


def sigmoid(x):
    return 1.0 / (1.0 + np.exp(-x))


def silu(z):
    return z * sigmoid(z)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + np.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def exact(x):
    return x


def dense_ff(h, gate, up, down, r=exact, act=gelu_tanh):
    return r(act(h @ gate.T) * (h @ up.T)) @ down.T


def soft_cap(x, cap):
    return cap * np.tanh(x / cap)


def log_sigmoid(x):
    return -np.logaddexp(0.0, -x)


def mlstm_cell(q, k, v, log_i, log_f, state):
    """One head of the matrix memory over T tokens. q (scaled), k: [T, dim]; v: [T, vdim]; state =
    (S [dim, vdim], n [dim], m), returned updated. The stabiliser m starts at 0."""
    S, n, m = state
    out = np.empty((len(q), v.shape[1]))
    for t in range(len(q)):
        m_new = max(log_f[t] + m, log_i[t])
        keep, take = math.exp(log_f[t] + m - m_new), math.exp(log_i[t] - m_new)
        S = keep * S + take * np.outer(k[t], v[t])
        n = keep * n + take * k[t]
        m = m_new
        out[t] = (S.T @ q[t]) / (max(abs(float(n @ q[t])), math.exp(-m)) + 1e-6)
    return out, (S, n, m)


def mlstm_mixer(h, w, p, mx, eps, state, r=exact):
    """state: list of per-head cell states or None for a new sequence. r: see Run."""
    H, d, dv, cap = mx["heads"], mx["dim"], mx["vdim"], mx["gate_cap"]
    T = len(h)
    q = r(h @ w[p + "q"].T).reshape(T, H, d) * d ** -0.5
    k = r(h @ w[p + "k"].T).reshape(T, H, d)
    v = r(h @ w[p + "v"].T).reshape(T, H, dv)
    li = soft_cap(h @ w[p + "i"].T + w[p + "i.b"], cap)
    lf = log_sigmoid(soft_cap(h @ w[p + "f"].T + w[p + "f.b"], cap))
    state = state or [(np.zeros((d, dv)), np.zeros(d), 0.0) for _ in range(H)]
    out, new = np.empty((T, H, dv)), []
    for a in range(H):
        out[:, a], s = mlstm_cell(q[:, a], k[:, a], v[:, a], li[:, a], lf[:, a], state[a])
        new.append(s)
    out = r(rms(out, eps).reshape(T, H * dv) * w[p + "norm"] * sigmoid(r(h @ w[p + "g"].T)))
    return out @ w[p + "o"].T, new


def rope_interleaved(x, pos, dims, base, factor):
    """x [..., dim] at position pos: pairs (2i, 2i+1) of the first `dims` dimensions turned."""
    y = np.array(x, dtype=np.float64)
    for i in range(dims // 2):
        a = pos * base ** (-2.0 * i / dims) / factor
        u, v = x[..., 2 * i], x[..., 2 * i + 1]
        y[..., 2 * i] = u * math.cos(a) - v * math.sin(a)
        y[..., 2 * i + 1] = v * math.cos(a) + u * math.sin(a)
    return y


def visible(i, j, size, keep_first):
    """What position i may look at: its window (size 0: everything before it) and the sequence's start."""
    return j <= i and (not size or i - j < size or j < keep_first)


def attend(q, keys, values, i, scale, size, keep_first):
    """Softmax average of the values that position i sees."""
    js = [j for j in range(len(keys)) if visible(i, j, size, keep_first)]
    s = np.array([float(q @ keys[j]) * scale for j in js])
    e = np.exp(s - s.max())
    return (e / e.sum()) @ values[js]


def diff_lambda(lq1, lk1, lq2, lk2, diff):
    return math.exp(float(np.sum(lq1 * lk1))) - math.exp(float(np.sum(lq2 * lk2))) + diff


def diff_attention_mixer(h, w, p, mx, eps, cache, r=exact):
    """cache: (list of keys [G, 2, dim], list of values [G, vdim]) or None; one entry a position."""
    H, G, d, dv = mx["heads"], mx["kv_heads"], mx["dim"], mx["vdim"]
    rot, mask = mx["rot"], mx.get("mask") or {}
    factor = (rot.get("scaling") or {}).get("factor", 1.0)
    K, V = ([], []) if cache is None else (list(cache[0]), list(cache[1]))
    T = len(h)
    q = r(h @ w[p + "q"].T).reshape(T, H, 2, d)
    k = r(h @ w[p + "k"].T).reshape(T, G, 2, d)
    v = r(h @ w[p + "v"].T).reshape(T, G, dv)
    lam = diff_lambda(*(np.asarray(w[p + n], np.float64) for n in ("lq1", "lk1", "lq2", "lk2")), mx["diff"])
    gate = sigmoid(h @ w[p + "g"].T)
    out = np.empty((T, H, dv))
    for t in range(T):
        i = len(K)
        K.append(r(rope_interleaved(k[t], i, rot["dims"], rot["base"], factor)))
        V.append(v[t])
        qr = r(rope_interleaved(q[t], i, rot["dims"], rot["base"], factor))
        Ka, Va = np.array(K), np.array(V)
        for a in range(H):
            g = a // (H // G)
            a1, a2 = (attend(qr[a, n], Ka[:, g, n], Va[:, g], i, mx["scale"], mask.get("size", 0),
                             mask.get("keep_first", 0)) for n in (0, 1))
            o = rms(a1 - lam * a2, eps) * (1.0 - mx["diff"])
            out[t, a] = o * gate[t, a]
    return r(out.reshape(T, H * dv)) @ w[p + "o"].T, (K, V)


def turn_frequencies(dims, base, scaling=None):
    """Angle per position of every pair, and what cos and sin are multiplied by. scaling: none, or YaRN's
    {factor, original, fast, slow} (Peng et al., "YaRN: Efficient Context Window Extension of Large
    Language Models"): pairs that turn often keep their frequency, slow ones get a `factor`-th of it."""
    f = np.array([base ** (-2.0 * i / dims) for i in range(dims // 2)])
    if not scaling:
        return f, 1.0
    pair_of = lambda turns: dims * math.log(scaling["original"] / (2 * math.pi * turns)) / (2 * math.log(base))
    lo, hi = max(math.floor(pair_of(scaling["fast"])), 0), min(math.ceil(pair_of(scaling["slow"])), dims - 1)
    slow = np.clip((np.arange(dims // 2) - lo) / max(hi - lo, 0.001), 0.0, 1.0)
    return f * (1 - slow) + f / scaling["factor"] * slow, 0.1 * math.log(scaling["factor"]) + 1.0


def turn(x, pos, freqs, gain, halves):
    """x [..., dim] at position pos; a pair is (2i, 2i+1), or with halves (i, i + n), n pairs in all."""
    y, n = np.array(x, dtype=np.float64), len(freqs)
    for i in range(n):
        a, b = (i, i + n) if halves else (2 * i, 2 * i + 1)
        c, s = gain * math.cos(pos * freqs[i]), gain * math.sin(pos * freqs[i])
        u, v = x[..., a], x[..., b]
        y[..., a] = u * c - v * s
        y[..., b] = v * c + u * s
    return y


def retention_cell(q, k, v, decay, S):
    """One head: S [dim, vdim] fades by `decay` a token, takes k v^T and is read along q."""
    out = np.empty((len(q), v.shape[1]))
    for t in range(len(q)):
        S = decay * S + np.outer(k[t], v[t])
        out[t] = S.T @ q[t]
    return out, S


def retention_mixer(h, w, p, mx, eps, cache, r=exact):
    """cache: (tokens seen, one S a head) or None."""
    H, d, dv = mx["heads"], mx["dim"], mx["vdim"]
    T = len(h)
    at, states = cache or (0, [np.zeros((d, dv)) for _ in range(H)])
    q = r(h @ w[p + "q"].T).reshape(T, H, d)
    k = r(h @ w[p + "k"].T).reshape(T, H, d)
    v = r(h @ w[p + "v"].T).reshape(T, H, dv)
    freqs, gain = turn_frequencies(mx["rot"]["dims"], mx["rot"]["base"], mx["rot"].get("scaling"))
    q = np.array([turn(q[t], at + t, freqs, gain, True) for t in range(T)])
    k = np.array([turn(k[t], at + t, freqs, gain, True) for t in range(T)]) * d ** -0.5
    out, new = np.empty((T, H, dv)), []
    for a in range(H):
        out[:, a], S = retention_cell(q[:, a], k[:, a], v[:, a], mx["decay"][a], states[a])
        new.append(S)
    out = r(rms(out, eps).reshape(T, H * dv) * silu(r(h @ w[p + "g"].T)))
    return out @ w[p + "o"].T, (at + T, new)


def attend_sink(scores, values, sink):
    """Softmax average of the values, exp(sink) in the denominator beside the scores' exponentials."""
    top = max(float(np.max(scores)), sink)
    e = np.exp(scores - top)
    return (e @ values) / (e.sum() + math.exp(sink - top))


def latent_attention_mixer(h, w, p, mx, eps, cache, r=exact, shared=None):
    """cache, shared: (list of latents [rank], list of turned key parts [rot_dim]); `shared` is that of the layer
    whose keys and values this one reads (its own stays None then)."""
    H, d, dr, dv, rank = mx["heads"], mx["dim"], mx["rot_dim"], mx["vdim"], mx["kv_rank"]
    T, size = len(h), (mx.get("mask") or {}).get("size", 0)
    freqs, gain = turn_frequencies(dr, mx["rot"]["base"], mx["rot"].get("scaling"))
    q = r(h @ w[p + "q"].T).reshape(T, H, d + dr)
    if shared is None:
        C, K = ([], []) if cache is None else (list(cache[0]), list(cache[1]))
        at, down = len(C), h @ w[p + "dkv"].T
        for t in range(T):
            C.append(r(norm_plain(down[t, :rank], w[p + "dkv.norm"], eps)))
            K.append(r(turn(down[t, rank:], at + t, freqs, gain, False)))
        cache = (C, K)
    else:
        (C, K), at = shared, len(shared[0]) - T
    gate = sigmoid(h @ w[p + "g"].T)
    out = np.empty((T, H, dv))
    for t in range(T):
        i = at + t
        js = [j for j in range(len(C)) if visible(i, j, size, 0)]
        c, kr = np.array([C[j] for j in js]), np.array([K[j] for j in js])
        qr = r(turn(q[t, :, d:], i, freqs, gain, False))
        for a in range(H):
            keys = c @ w[p + "uk"][a * d:(a + 1) * d].T
            vals = c @ w[p + "uv"][a * dv:(a + 1) * dv].T
            s = (keys @ q[t, a, :d] + kr @ qr[a]) * mx["scale"]
            out[t, a] = attend_sink(s, vals, float(w[p + "sink"][a])) * gate[t, a]
    return r(out.reshape(T, H * dv)) @ w[p + "o"].T, cache if shared is None else None


MIXERS = {"mlstm": mlstm_mixer, "attention": diff_attention_mixer, "retention": retention_mixer,
          "latent_attention": latent_attention_mixer}


class Run:
    """One sequence through the model; feed() takes its next tokens and returns the logits at each.
    r: what happens to every activation that is stored between operations (nothing; a rounding or a
    disturbance of its size, to learn what it does to the logits)."""

    def __init__(self, cfg, w, r=exact):
        self.r = r
        self.cfg, self.w = cfg, {n: np.asarray(a, np.float64) for n, a in w.items()}
        self.state = [None] * len(cfg["layers"])

    def mix(self, i, h):
        layer, kw = self.cfg["layers"][i], {}
        if layer["mixer"].get("kv_from") is not None:
            kw["shared"] = self.state[layer["mixer"]["kv_from"]]
        y, self.state[i] = MIXERS[layer["type"]](h, self.w, f"l{i}.mix.", layer["mixer"], self.cfg["norm"]["eps"],
                                                 self.state[i], self.r, **kw)
        return y

    def ff(self, i, h, act):
        p = f"l{i}.mlp."
        return dense_ff(h, self.w[p + "gate"], self.w[p + "up"], self.w[p + "down"], self.r, act)

    def feed(self, tokens, trail=None):
        """trail: a list that receives the residual stream after every layer."""
        run = {"Pigodra": self._one_after_the_other, "Ranavik": self._side_by_side}[self.cfg["architecture"]]
        return run(self.w["embed"][np.asarray(tokens)], trail)

    def _one_after_the_other(self, x, trail):
        cfg, w, eps = self.cfg, self.w, self.cfg["norm"]["eps"]
        x = x * cfg["embedding"]["scale"]
        for i, layer in enumerate(cfg["layers"]):
            p = f"l{i}."
            x = x + self.mix(i, self.r(norm_zero_centred(x, w[p + "norm1"], eps)))
            if layer["mlp"] is not None:
                x = x + self.ff(i, self.r(norm_zero_centred(x, w[p + "norm2"], eps)), gelu_tanh)
            if trail is not None:
                trail.append(x)
        self.hidden = self.r(norm_zero_centred(x, w["final.norm"], eps))
        return self.hidden @ w["head"].T

    def _side_by_side(self, x, trail):
        """Mixer and feed-forward read the same stream; their sum goes back times residual_mult."""
        cfg, w, eps = self.cfg, self.w, self.cfg["norm"]["eps"]
        x = norm_plain(x, w["embed.norm"], eps)
        for i, layer in enumerate(cfg["layers"]):
            p = f"l{i}."
            y = self.mix(i, self.r(norm_plain(x, w[p + "norm1"], eps)))
            if layer["mlp"] is not None:
                y = y + self.ff(i, self.r(norm_plain(x, w[p + "norm2"], eps)), silu)
            x = x + cfg["residual_mult"] * y
            if trail is not None:
                trail.append(x)
        self.hidden = self.r(norm_plain(x, w["final.norm"], eps))
        return soft_cap(self.hidden @ w["head"].T, cfg["logit_softcap"])
