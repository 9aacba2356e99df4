"""CPU: the NumPy statement of the Rirotar decoder (oracle/rirotar_oracle.py) against closed forms and second spellings of its
mechanisms, so that the GPU tests compare the library with something that has itself been pinned."""
import math

import numpy as np

from oracle import rirotar_oracle as O
from tests import rirotar_util as U


def test_norm_weight_is_stored_around_zero_and_eps_sits_inside_the_root():
    x = np.array([[3.0, -4.0]])
    assert np.allclose(O.layer_norm1p(x, np.array([0.0, 1.0]), 0.0), x / math.sqrt(12.5) * [1.0, 2.0])
    assert np.allclose(O.unit_rms(np.full((1, 4), 2.0), 5.0), 2.0 / 3.0)
    assert np.allclose(O.unit_length(np.array([[3.0, 4.0]])), [[0.6, 0.8]], atol=1e-6)


def test_window_sees_itself_and_the_tokens_before_it_and_the_sink_takes_its_share():
    p = O.window_softmax_with_sink(np.zeros((9, 9)), math.log(2.0), 3)
    for i in range(9):
        seen = np.nonzero(p[i])[0]
        assert list(seen) == list(range(max(0, i - 2), i + 1))
        assert np.allclose(p[i, seen], 1.0 / (len(seen) + 2.0))
    assert np.allclose(O.window_softmax_with_sink(np.zeros((4, 4)), -1e9, 1), np.eye(4))
    big = O.window_softmax_with_sink(np.full((2, 2), 700.0), 701.0, 5)                 # no overflow; the sink is larger than every score
    assert np.allclose(big[1], 1.0 / (2.0 + math.e))


def test_latent_attention_as_explicit_sums_and_in_the_latent_space():
    rs = np.random.RandomState(1)
    mx = U.latent(heads=2, dim=3, vdim=4, kv_rank=5, size=3, scale=0.7)
    cfg = U.config([U.layer("latent_attention", mx, None)], width=6)
    P = {k: v.astype(float) for k, v in U.random_weights(cfg, 1).items()}
    h, q = rs.randn(7, 6), "l0.mix."
    got = O.latent_attention(h, P, q, mx, 1e-5)
    lat = h @ P[q + "dkv"].T
    c = lat / np.sqrt((lat ** 2).mean(-1, keepdims=True) + 1e-5) * P[q + "dkv.norm"]
    out = np.zeros((7, 8))
    for t in range(7):
        for hd in range(2):
            qh = P[q + "q"][3 * hd:3 * hd + 3] @ h[t]
            lat_q = P[q + "uk"][3 * hd:3 * hd + 3].T @ qh                                # the same scores against the latent itself
            js = range(max(0, t - 2), t + 1)
            w = np.array([math.exp(0.7 * lat_q @ c[j]) for j in js])
            w /= w.sum() + math.exp(P[q + "sink"][hd])
            out[t, 4 * hd:4 * hd + 4] = P[q + "uv"][4 * hd:4 * hd + 4] @ sum(wj * c[j] for wj, j in zip(w, js))
    assert np.allclose(got, out @ P[q + "o"].T)


def test_convolution_columns_and_zeros_in_front():
    x = np.arange(1.0, 6.0)[:, None]
    assert np.allclose(O.causal_conv(x, np.array([[0.0, 0.0, 1.0]])), x)
    assert np.allclose(O.causal_conv(x, np.array([[1.0, 0.0, 0.0]]))[:, 0], [0, 0, 1, 2, 3])
    assert np.allclose(O.causal_conv(x, np.array([[2.0]])), 2 * x)


def test_delta_rule_writes_what_is_missing():
    T, d, e = 5, 4, 3
    rs = np.random.RandomState(2)
    q = np.tile(np.eye(d)[0], (T, 1, 1)).reshape(T, 1, d)
    v = rs.randn(T, 1, e)
    one = np.ones((T, 1))
    # full write strength, no decay, the same key every time: the state holds the newest value, read in the same step
    assert np.allclose(O.delta_rule(q, q, v, one, np.zeros((T, 1))), v)
    # half strength: an exponential average
    want, s = [], np.zeros(e)
    for t in range(T):
        s = s + 0.5 * (v[t, 0] - s)
        want.append(s.copy())
    assert np.allclose(O.delta_rule(q, q, v, 0.5 * one, np.zeros((T, 1)))[:, 0], want)
    # orthogonal keys do not disturb each other; the decay acts before the write
    k = np.eye(d)[[0, 1, 2, 3, 1]].reshape(T, 1, d)
    o = O.delta_rule(np.ones((T, 1, d)), k, v, one, np.full((T, 1), math.log(0.5)))
    assert np.allclose(o[3, 0], sum(0.5 ** (3 - t) * v[t, 0] for t in range(4)))
    assert np.allclose(o[4, 0], v[4, 0] + sum(0.5 ** (4 - t) * v[t, 0] for t in (0, 2, 3)))


def test_delta_rule_as_a_triangular_system():
    """The same outputs without a state: (I + A) U = beta V, o_t = sum_(s <= t) P[t][s] u_s, decays per key channel."""
    rs = np.random.RandomState(3)
    T, H, G, d, e = 9, 4, 2, 5, 3
    q, k = rs.randn(T, G, d), O.unit_length(rs.randn(T, G, d))
    v, beta, ld = rs.randn(T, H, e), rs.rand(T, H), -rs.rand(T, H, d)
    got = O.delta_rule(q, k, v, beta, ld)
    b = np.cumsum(ld, 0)
    for h in range(H):
        g = h // 2
        A, Pm = np.zeros((T, T)), np.zeros((T, T))
        for t in range(T):
            for s in range(t + 1):
                f = np.exp(b[t, h] - b[s, h])
                Pm[t, s] = (q[t, g] * k[s, g] * f).sum()
                if s < t:
                    A[t, s] = beta[t, h] * (k[t, g] * k[s, g] * f).sum()
        u = np.linalg.solve(np.eye(T) + A, beta[:, h, None] * v[:, h])
        assert np.allclose(got[:, h], Pm @ u)
    # one number per head is the same as that number on every key channel
    ldh = -rs.rand(T, H)
    assert np.allclose(O.delta_rule(q, k, v, beta, ldh), O.delta_rule(q, k, v, beta, np.repeat(ldh[:, :, None], d, 2)))


def test_channel_decay_with_equal_rows_is_the_head_decay():
    mx = U.delta(heads=2, kv_heads=2, dim=4, vdim=6, conv=2)
    cfg = U.config([U.layer("channel_delta", mx, None)], width=8)
    P = {k: v.astype(float) for k, v in U.random_weights(cfg, 4, (3, 5)).items()}
    q = "l0.mix."
    P[q + "a2"] = np.repeat(P[q + "a2"].reshape(2, 4, 3)[:, :1], 4, 1).reshape(8, 3)
    P[q + "dt_bias"] = np.repeat(P[q + "dt_bias"].reshape(2, 4)[:, :1], 4, 1).reshape(8)
    h = np.random.RandomState(4).randn(6, 8)
    ch = O.channel_log_decay(h, P, q, mx)
    P[q + "a"] = P[q + "a2"].reshape(2, 4, 3)[:, 0] @ P[q + "a1"]
    P[q + "dt_bias"] = P[q + "dt_bias"].reshape(2, 4)[:, 0]
    assert np.allclose(ch, O.head_log_decay(h, P, q, mx)[:, :, None]) and (ch < 0).all()


def test_gates_of_the_two_delta_kinds():
    rs = np.random.RandomState(5)
    for kind, gate in (("delta", lambda P, h: O.silu(h @ P["l0.mix.g"].T)), ("channel_delta", lambda P, h: O.sigmoid(h @ P["l0.mix.g1"].T @ P["l0.mix.g2"].T))):
        mx = U.delta(heads=2, kv_heads=1, dim=4, vdim=6, conv=3)
        cfg = U.config([U.layer(kind, mx, None)], width=8)
        P = {k: v.astype(float) for k, v in U.random_weights(cfg, 5).items()}
        h = rs.randn(7, 8)
        qq, kk, vv, beta = O.delta_inputs(h, P, "l0.mix.", mx)
        assert np.allclose((kk ** 2).sum(-1), 1.0, atol=1e-3) and np.allclose((qq ** 2).sum(-1), 0.25, atol=1e-3)
        ld = (O.head_log_decay if kind == "delta" else O.channel_log_decay)(h, P, "l0.mix.", mx)
        o = O.delta_rule(qq, kk, vv, beta, ld)
        y = o / np.sqrt((o ** 2).mean(-1, keepdims=True) + 1e-6) * P["l0.mix.norm"]
        assert np.allclose(O.MIXERS[kind](h, P, "l0.mix.", mx, 1e-6), (y.reshape(7, 12) * gate(P, h)) @ P["l0.mix.o"].T)


def test_caps_of_the_feed_forward():
    P = {"gate": np.array([[1.0]]), "up": np.array([[1.0]]), "down": np.array([[1.0]])}
    f = lambda x, lim: float(O.capped_ff(np.array([[x]]), P, "", lim)[0, 0])
    assert np.isclose(f(0.5, 2.0), 0.5 / (1 + math.exp(-0.851)) * 1.5)
    assert np.isclose(f(9.0, 2.0), 2.0 / (1 + math.exp(-3.404)) * 3.0)                  # both capped
    assert np.isclose(f(-9.0, 2.0), -9.0 / (1 + math.exp(1.702 * 9.0)) * -1.0)          # the gate has no lower cap


def test_router_groups_by_the_sum_of_their_two_best_and_scales_the_weights():
    logit = lambda s: math.log(s / (1 - s))
    # group 0 holds the largest score, groups 1 and 2 the larger sums
    s = np.array([0.9, 0.05, 0.1, 0.6, 0.55, 0.1, 0.5, 0.58, 0.2])
    P = {"router": np.array([[logit(x)] for x in s])}
    rt = dict(experts=9, top=3, groups=dict(count=3, keep=2), scale=2.0)
    sel, w = O.route(np.array([[1.0]]), P, "", rt)
    assert list(sel[0]) == [3, 7, 4]
    assert np.allclose(w[0], 2.0 * np.array([0.6, 0.58, 0.55]) / 1.73)
    sel, _ = O.route(np.array([[1.0]]), P, "", dict(rt, groups=dict(count=3, keep=3)))
    assert list(sel[0]) == [0, 3, 7]
    sel, _ = O.route(np.array([[1.0]]), P, "", dict(rt, groups=dict(count=9, keep=3)))  # one expert per group
    assert list(sel[0]) == [0, 3, 7]
    sel, _ = O.route(np.array([[1.0]]), P, "", dict(rt, groups=dict(count=1, keep=1)))
    assert list(sel[0]) == [0, 3, 7]


def test_logits_stay_inside_the_cap_and_the_model_is_causal():
    cfg = U.small_config()
    P = U.random_weights(cfg, 6)
    toks = U.tokens(30, cfg["vocab"], 6)
    a = O.forward(cfg, P, toks)
    assert np.abs(a).max() < cfg["logit_softcap"]
    other = list(toks)
    other[20] = (toks[20] + 1) % cfg["vocab"]
    b = O.forward(cfg, P, other)
    assert np.allclose(a[:20], b[:20]) and not np.allclose(a[20:], b[20:])
    loose = dict(cfg, logit_softcap=1e6)
    raw = O.forward(loose, P, toks)
    assert np.allclose(a, 9.0 * np.tanh(raw / 9.0), atol=1e-4)


def test_planted_key_shows_exactly_inside_the_window():
    cfg, P, QT, KT = U.planted_window(5)
    for dist in (4, 5):
        toks = U.tokens(12, 65, dist)
        toks[3], toks[3 + dist] = KT, QT
        plain = list(toks)
        plain[3] = 1
        a, b = O.forward(cfg, P, toks)[3 + dist], O.forward(cfg, P, plain)[3 + dist]
        moved = np.abs(a - b).max() / np.abs(a).max()
        assert (moved > 0.1) == (dist < 5) and (dist < 5 or moved < 1e-9)
