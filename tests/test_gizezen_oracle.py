"""CPU: the NumPy statement of the Gizezen decoder (oracle/gizezen_oracle.py) against closed forms and second spellings of its
mechanisms, so that the GPU tests compare the library with something that has itself been pinned."""
import math

import numpy as np
import pytest

from oracle import gizezen_oracle as O
from tests import gizezen_util as U


def test_norm_works_element_by_element():
    P = {"n": np.array([2.0, -1.0, 3.0]), "n.b": np.array([0.5, 0.0, -1.0]), "n.alpha": np.array(0.25)}
    x = np.array([[4.0, -8.0, 0.0], [0.0, 0.0, 400.0]])
    t = math.tanh
    assert np.allclose(O.tanh_norm(x, P, "n"), [[2 * t(1) + 0.5, t(2), -1.0], [0.5, 0.0, 2.0]])
    assert np.allclose(O.tanh_norm(x[:, :1], dict(P, n=P["n"][:1], **{"n.b": P["n.b"][:1]}), "n"), O.tanh_norm(x, P, "n")[:, :1])    # no statistic of the row


def test_convolution_taps_run_from_the_oldest_to_the_current_token():
    x = np.array([[1.0], [10.0], [100.0], [1000.0]])
    assert np.allclose(O.causal_conv(x, np.array([[3.0, 2.0, 1.0]]))[:, 0], [1, 12, 123, 1230])
    assert np.allclose(O.causal_conv(x, np.array([[5.0]])), 5 * x)


def test_frequencies_are_kept_stretched_or_blended_by_wavelength():
    rot = dict(base=10000.0, dims=16)
    f = O.frequencies(rot)
    assert np.allclose(f, [10000.0 ** (-i / 8) for i in range(8)])
    assert O.frequencies(dict(rot, scaling=None)).tolist() == f.tolist()
    sc = dict(factor=4.0, low=1.0, high=4.0, original=200)
    g = O.frequencies(dict(rot, scaling=sc))
    wl = 2 * np.pi / f
    kinds = set()
    for i in range(8):
        if wl[i] < 50:
            kinds.add("kept"); assert g[i] == f[i]
        elif wl[i] > 200:
            kinds.add("stretched"); assert np.isclose(g[i], f[i] / 4)
        else:
            kinds.add("blended"); assert f[i] / 4 < g[i] < f[i]
            s = (200 / wl[i] - 1) / 3
            assert np.isclose(g[i], f[i] * ((1 - s) / 4 + s))
    assert kinds == {"kept", "stretched", "blended"}
    # the blend meets both sides at its ends
    for edge, ratio in ((50.0, 1.0), (200.0, 0.25)):
        base = (edge * (1 + 1e-12) / (2 * np.pi)) ** (4 / 2)          # pair 1 of 2: wavelength = edge
        r = dict(base=base, dims=4, scaling=sc)
        assert np.isclose(O.frequencies(r)[1] / base ** -0.5, ratio, atol=1e-9)


def test_rotation_turns_neighbours_and_leaves_the_rest():
    rs = np.random.RandomState(0)
    x = rs.randn(9, 2, 7)
    rot = dict(base=50.0, dims=4)
    y = O.rotate(x, rot)
    assert np.array_equal(y[..., 4:], x[..., 4:]) and np.allclose(y[0], x[0])
    for i in range(2):
        z = (x[..., 2 * i] + 1j * x[..., 2 * i + 1]) * np.exp(1j * np.arange(9) * 50.0 ** (-i / 2))[:, None]
        assert np.allclose(y[..., 2 * i], z.real) and np.allclose(y[..., 2 * i + 1], z.imag)
    assert np.array_equal(O.rotate(x, dict(base=50.0, dims=0)), x) and np.array_equal(O.rotate(x, None), x)
    # scores depend on the distance alone
    q = np.repeat(x[:1], 9, 0)
    s = np.einsum("ihd,jhd->hij", O.rotate(q, rot), O.rotate(q, rot))
    assert np.allclose(s[:, 3, 1], s[:, 8, 6])


def test_window_and_the_one_in_the_denominator():
    p = O.window_softmax_plus_one(np.zeros((9, 9)), 3)
    for i in range(9):
        seen = np.nonzero(p[i])[0]
        assert list(seen) == list(range(max(0, i - 2), i + 1))
        assert np.allclose(p[i, seen], 1.0 / (len(seen) + 1.0))
    z = np.log(np.array([[2.0, 9.0], [3.0, 5.0]]))
    assert np.allclose(O.window_softmax_plus_one(z, 5), [[2 / 3, 0], [3 / 9, 5 / 9]])
    assert np.allclose(O.window_softmax_plus_one(np.full((2, 2), 800.0), 5)[1], 0.5)          # no overflow
    assert np.allclose(O.window_softmax_plus_one(np.full((2, 2), -800.0), 5), 0.0)            # the one takes everything


def test_queries_and_keys_have_unit_root_mean_square_after_the_rotation():
    mx = U.attn(heads=3, kv_heads=1, dim=10, rot_dims=6, conv=2)
    cfg = U.config([U.layer(mx, None)], width=8)
    P = U.random_weights(cfg, 1)
    h = np.random.RandomState(1).randn(6, 8)
    q = O.queries_or_keys(h, P, "l0.mix.q", 3, mx, 0.0)
    assert np.allclose((q ** 2).mean(-1), 1.0)
    # a rotation of a part and a division by the whole head's length commute (the same length) -- an offset in between would not
    raw = O.causal_conv(h @ P["l0.mix.q"].astype(float).T, P["l0.mix.q.conv"]).reshape(6, 3, 10)
    assert np.allclose(O.rotate(raw / np.sqrt((raw ** 2).mean(-1, keepdims=True)), mx["rot"]), q)
    assert np.allclose(O.unit_rms(np.full((1, 4), 2.0), 5.0), 2.0 / 3.0)                      # eps inside the root
    v = O.keys_and_values(h, P, "l0.mix.", mx, 0.0)[1]
    assert np.allclose(v[:, 0], O.causal_conv(h @ P["l0.mix.v"].astype(float).T, P["l0.mix.v.conv"]))         # neither rotated nor normed


def test_attention_as_explicit_sums_with_gate_and_shared_key_heads():
    rs = np.random.RandomState(2)
    mx = U.attn(heads=4, kv_heads=2, dim=3, vdim=5, conv=2, size=3, scale=0.7, rot_dims=2)
    cfg = U.config([U.layer(mx, None)], width=6)
    P = {k: v.astype(float) for k, v in U.random_weights(cfg, 2).items()}
    h, pre = rs.randn(7, 6), "l0.mix."
    k, v = O.keys_and_values(h, P, pre, mx, 1e-5)
    q = O.queries_or_keys(h, P, pre + "q", 4, mx, 1e-5)
    got = O.attention(h, P, pre, mx, 1e-5, (k, v))
    out = np.zeros((7, 20))
    for t in range(7):
        for hd in range(4):
            js = range(max(0, t - 2), t + 1)
            w = [math.exp(0.7 * float(q[t, hd] @ k[j, hd // 2])) for j in js]
            o = sum(wi * v[j, hd // 2] for wi, j in zip(w, js)) / (1.0 + sum(w))
            out[t, hd * 5:hd * 5 + 5] = o / (1.0 + math.exp(-float(P[pre + "g"][hd] @ h[t])))
    assert np.allclose(got, out @ P[pre + "o"].T)


def test_borrowed_keys_are_the_other_layers_and_everything_else_is_its_own():
    lend, borrow = U.attn(size=4, rot_dims=8), U.attn(heads=2, size=9, conv=4, rot_dims=4, kv_from=0)
    cfg = U.config([U.layer(lend, None), U.layer(borrow, None)])
    P = U.random_weights(cfg, 3)
    assert "l1.mix.k" not in P and "l1.mix.v.conv" not in P and "l1.mix.q.conv" in P
    toks = U.tokens(14, cfg["vocab"], 3)
    x = P["embed"].astype(float)[toks] * cfg["embedding"]["scale"]
    h0 = O.tanh_norm(x, P, "l0.norm1")
    kv = O.keys_and_values(h0, P, "l0.mix.", lend, cfg["norm"]["eps"])
    x = x + 0.4 * O.attention(h0, P, "l0.mix.", lend, cfg["norm"]["eps"], kv)
    x = x + 0.4 * O.attention(O.tanh_norm(x, P, "l1.norm1"), P, "l1.mix.", borrow, cfg["norm"]["eps"], kv)
    _, rows = O.forward(cfg, P, toks, True)
    assert np.allclose(rows[-1], x)


def test_router_takes_the_largest_logits_and_the_softmax_over_them_alone():
    z = np.array([0.3, 2.0, -1.0, 1.5, 1.9])
    P = {"router": z[:, None]}
    sel, w = O.route(np.array([[1.0]]), P, "", dict(experts=5, top=3))
    assert list(sel[0]) == [1, 4, 3]
    e = np.exp([2.0, 1.9, 1.5])
    assert np.allclose(w[0], e / e.sum())
    full = np.exp(z) / np.exp(z).sum()                               # the same as the softmax over all, divided by the chosen ones' sum
    assert np.allclose(w[0], full[[1, 4, 3]] / full[[1, 4, 3]].sum())
    sel, w = O.route(np.array([[1000.0]]), P, "", dict(experts=5, top=1))
    assert list(sel[0]) == [1] and w[0, 0] == 1.0


def test_mixture_as_explicit_sums_and_the_gated_shared_expert():
    ml = U.moe(experts=4, top=2, ff=5, shared=7)
    cfg = U.config([U.layer(U.attn(), ml)], width=6)
    P = {k: v.astype(float) for k, v in U.random_weights(cfg, 4).items()}
    h, pre = np.random.RandomState(4).randn(5, 6), "l0.mlp."
    ff = lambda x, n: P[n + "down"] @ ((lambda g: g / (1 + np.exp(-g)))(P[n + "gate"] @ x) * (P[n + "up"] @ x))
    want = []
    for x in h:
        z = P[pre + "router"] @ x
        a, b = np.argsort(-z)[:2]
        wa = 1 / (1 + math.exp(z[b] - z[a]))
        sg = 1 / (1 + math.exp(-float(P[pre + "shared.sg"][0] @ x)))
        want.append(wa * ff(x, f"{pre}e{a}.") + (1 - wa) * ff(x, f"{pre}e{b}.") + sg * ff(x, pre + "shared."))
    assert np.allclose(O.mixture_ff(h, P, pre, ml), want)
    alone = dict(ml); del alone["shared"]
    gate = 1 / (1 + np.exp(-h @ P[pre + "shared.sg"].T))
    assert np.allclose(O.mixture_ff(h, P, pre, ml) - O.mixture_ff(h, P, pre, alone), gate * np.array([ff(x, pre + "shared.") for x in h]))


def test_embedding_scale_residual_multiplier_and_causality():
    cfg = U.small_config()
    P = U.random_weights(cfg, 5)
    toks = U.tokens(30, cfg["vocab"], 5)
    a, rows = O.forward(cfg, P, toks, True)
    still, srows = O.forward(dict(cfg, residual_mult=0.0), P, toks, True)
    assert np.allclose(srows[-1], 2.5 * P["embed"].astype(float)[toks])
    assert np.allclose(still, O.tanh_norm(srows[-1], P, "final.norm") @ P["head"].astype(float).T)
    other = list(toks)
    other[20] = (toks[20] + 1) % cfg["vocab"]
    b = O.forward(cfg, P, other)
    assert np.allclose(a[:20], b[:20]) and not np.allclose(a[20:], b[20:])


@pytest.mark.parametrize("size,borrowed", [(5, None), (20, None), (5, 9), (9, 5)])
def test_planted_key_shows_exactly_inside_the_window(size, borrowed):
    cfg, P, QT, KT = U.planted_window(size, borrowed)
    edge = borrowed or size
    for dist in (1, edge - 1, edge, edge + 1):
        toks = U.tokens(40, 65, dist)
        toks[3], toks[3 + dist] = KT, QT
        plain = list(toks)
        plain[3] = 1
        a, b = O.forward(cfg, P, toks)[3 + dist], O.forward(cfg, P, plain)[3 + dist]
        moved = np.abs(a - b).max() / np.abs(a).max()
        assert (moved > 0.1) == (dist < edge) and (dist < edge or moved < 1e-9), (dist, moved)
