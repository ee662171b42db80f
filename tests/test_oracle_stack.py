"""CPU: the plain reference of the layer-list designs (tests/ref_stack.py) against closed forms and
second formulations of the same mathematics."""
import math

import numpy as np
import pytest

import ref_stack as R
import stack_models as M


def test_mlstm_cell_against_the_unstabilised_sums():
    """The running maximum only rescales: with S~ = sum of e^(F_t - F_s + i_s) k v^T the output is
    S~^T q / (max(|n~ . q|, 1) + 1e-6 e^m), m_t = max(F_t, max_s(F_t - F_s + i_s))."""
    rng = np.random.default_rng(0)
    T, d, dv = 40, 6, 5
    q, k, v = rng.standard_normal((T, d)), rng.standard_normal((T, d)), rng.standard_normal((T, dv))
    li, lf = 3 * rng.standard_normal(T), R.log_sigmoid(2 * rng.standard_normal(T) + 1)
    out, (S, n, m) = R.mlstm_cell(q, k, v, li, lf, (np.zeros((d, dv)), np.zeros(d), 0.0))
    F = np.cumsum(lf)
    for t in range(T):
        w = np.exp(F[t] - F[:t + 1] + li[:t + 1])
        top = max(F[t], float(np.max(F[t] - F[:t + 1] + li[:t + 1])))
        num = (w * (k[:t + 1] @ q[t])) @ v[:t + 1]
        den = float(np.sum(w * (k[:t + 1] @ q[t])))
        np.testing.assert_allclose(out[t], num / (max(abs(den), 1.0) + 1e-6 * math.exp(top)), rtol=1e-9, atol=1e-12)
    assert abs(m - top) < 1e-9


def test_mlstm_maximum_starts_at_zero():
    """With a first input gate far below zero the maximum stays at the decayed zero."""
    q = k = v = np.ones((1, 1))
    _, (_, _, m) = R.mlstm_cell(q, k, v, np.array([-9.0]), np.array([-0.5]), (np.zeros((1, 1)), np.zeros(1), 0.0))
    assert m == -0.5


def test_rotation_keeps_lengths_and_turns_by_distance():
    rng = np.random.default_rng(1)
    a, b = rng.standard_normal(12), rng.standard_normal(12)
    for p, s in ((0, 7), (3, 10), (900, 907)):
        ra, rb = R.rope_interleaved(a, p, 8, 500.0, 2.0), R.rope_interleaved(b, s, 8, 500.0, 2.0)
        assert abs(ra @ ra - a @ a) < 1e-9 and np.array_equal(ra[8:], a[8:])
        assert abs(ra @ rb - R.rope_interleaved(a, 0, 8, 500.0, 2.0) @ R.rope_interleaved(b, s - p, 8, 500.0, 2.0)) < 1e-9
    # factor 2 at position 2p is factor 1 at position p
    np.testing.assert_allclose(R.rope_interleaved(a, 18, 8, 500.0, 2.0), R.rope_interleaved(a, 9, 8, 500.0, 1.0), atol=1e-12)


@pytest.mark.parametrize("size,keep,i,seen", [(4, 0, 9, [6, 7, 8, 9]), (4, 2, 9, [0, 1, 6, 7, 8, 9]), (4, 2, 3, [0, 1, 2, 3]),
                                              (4, 8, 9, [0, 1, 2, 3, 4, 5, 6, 7, 8, 9]), (1, 0, 5, [5]), (0, 0, 3, [0, 1, 2, 3])])
def test_window_with_kept_first_tokens(size, keep, i, seen):
    assert [j for j in range(12) if R.visible(i, j, size, keep)] == seen


def test_attention_is_the_softmax_average():
    rng = np.random.default_rng(2)
    K, V, q = rng.standard_normal((9, 4)), rng.standard_normal((9, 3)), rng.standard_normal(4)
    w = np.exp(K[3:9] @ q * 0.3)
    np.testing.assert_allclose(R.attend(q, K, V, 8, 0.3, 6, 0), (w @ V[3:9]) / w.sum(), rtol=1e-12)


@pytest.mark.parametrize("name", sorted(M.CONFIGS))
def test_portions_do_not_matter(name):
    """The reference itself: a prompt at once, token by token and in uneven portions."""
    cfg = M.CONFIGS[name]
    w = M.weights(cfg, 3)
    toks = np.random.default_rng(4).integers(0, cfg["vocab"], 40)
    whole = R.Run(cfg, w).feed(toks)
    for cuts in ([1] * 40, [2, 2, 17, 3, 16]):
        run, at, got = R.Run(cfg, w), 0, []
        for n in cuts:
            got.append(run.feed(toks[at:at + n]))
            at += n
        np.testing.assert_allclose(np.concatenate(got), whole, rtol=1e-9, atol=1e-9)


def test_retention_against_the_sum_over_tokens():
    """o_t = sum_s decay^(t-s) (q_t . k_s) v_s."""
    rng = np.random.default_rng(5)
    T, d, dv = 30, 6, 5
    q, k, v = rng.standard_normal((T, d)), rng.standard_normal((T, d)), rng.standard_normal((T, dv))
    for g in (0.0, 0.9, 1.0):
        out, S = R.retention_cell(q, k, v, g, np.zeros((d, dv)))
        for t in range(T):
            w = np.array([g ** (t - s) for s in range(t + 1)]) * (k[:t + 1] @ q[t])
            np.testing.assert_allclose(out[t], w @ v[:t + 1], rtol=1e-9, atol=1e-12)
    np.testing.assert_allclose(S, k.T @ v, rtol=1e-9, atol=1e-12)


def test_turned_halves_are_turned_pairs_in_another_order():
    rng = np.random.default_rng(6)
    x, f = rng.standard_normal(11), R.turn_frequencies(8, 300.0)[0]
    order = [0, 4, 1, 5, 2, 6, 3, 7, 8, 9, 10]
    np.testing.assert_allclose(R.turn(x, 9, f, 1.0, True)[order], R.turn(x[order], 9, f, 1.0, False), rtol=1e-12)
    np.testing.assert_allclose(R.turn(x, 9, f, 1.0, False), R.rope_interleaved(x, 9, 8, 300.0, 1.0), rtol=1e-12)


def test_yarn_keeps_fast_pairs_and_stretches_slow_ones():
    sc = dict(factor=8.0, original=4096, fast=32.0, slow=1.0)
    f, gain = R.turn_frequencies(64, 1e4, sc)
    plain, one = R.turn_frequencies(64, 1e4)
    turns = 4096 * plain / (2 * math.pi)  # over the original positions
    assert one == 1.0 and abs(gain - (1 + 0.1 * math.log(8))) < 1e-12
    np.testing.assert_allclose(f[turns > 45], plain[turns > 45], rtol=1e-12)
    np.testing.assert_allclose(f[turns < 0.7], plain[turns < 0.7] / 8, rtol=1e-12)
    assert np.all(np.diff(f / plain) <= 1e-12)
    np.testing.assert_allclose(R.turn_frequencies(64, 1e4, dict(sc, factor=1.0))[0], plain, rtol=1e-12)


def test_a_sink_is_a_key_without_a_value():
    rng = np.random.default_rng(7)
    s, v = rng.standard_normal(5), rng.standard_normal((5, 3))
    e = np.exp(np.append(s, 0.7))
    np.testing.assert_allclose(R.attend_sink(s, v, 0.7), (e / e.sum()) @ np.vstack([v, np.zeros(3)]), rtol=1e-12)
