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


def sigmoid(x):
    return 1.0 / (1.0 + np.exp(-x))


def gelu_tanh(z):
    return 0.5 * z * (1.0 + np.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def exact(x):
    return x


def dense_ff(h, gate, up, down, r=exact):
    return r(gelu_tanh(h @ gate.T) * (h @ up.T)) @ down.T


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


MIXERS = {"mlstm": mlstm_mixer, "attention": diff_attention_mixer}


class Run:
    """One sequence through the model; feed() takes its next tokens and returns the logits at each.
    r: what happens to every activation that is stored between operations (nothing; a rounding or a
    disturbance of its size, to learn what it does to the logits)."""

    def __init__(self, cfg, w, r=exact):
        self.r = r
        self.cfg, self.w = cfg, {n: np.asarray(a, np.float64) for n, a in w.items()}
        self.state = [None] * len(cfg["layers"])

    def feed(self, tokens, trail=None):
        """trail: a list that receives the residual stream after every layer."""
        cfg, w, eps = self.cfg, self.w, self.cfg["norm"]["eps"]
        x = w["embed"][np.asarray(tokens)] * cfg["embedding"]["scale"]
        for i, layer in enumerate(cfg["layers"]):
            p = f"l{i}."
            y, self.state[i] = MIXERS[layer["type"]](self.r(norm_zero_centred(x, w[p + "norm1"], eps)), w, p + "mix.",
                                                     layer["mixer"], eps, self.state[i], self.r)
            x = x + y
            if layer["mlp"] is not None:
                x = x + dense_ff(self.r(norm_zero_centred(x, w[p + "norm2"], eps)), w[p + "mlp.gate"], w[p + "mlp.up"],
                                 w[p + "mlp.down"], self.r)
            if trail is not None:
                trail.append(x)
        self.hidden = self.r(norm_zero_centred(x, w["final.norm"], eps))
        return self.hidden @ w["head"].T
