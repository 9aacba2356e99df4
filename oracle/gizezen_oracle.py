"""Plain NumPy statement of the Gizezen decoder, one function per mechanism (float64, whole sequences, no cache).

Test infrastructure only: nothing here is imported by the product.  A model is a config dict in the checkpoint's own
spelling (``architecture``, ``width``, ``vocab``, ``embedding.scale``, ``residual_mult``, ``norm.eps``, ``layers[...]``) and a
dict of arrays under the checkpoint's tensor names (``embed``, ``l<i>.norm1``, ``l<i>.norm1.alpha``, ``l<i>.norm1.b``,
``l<i>.mix.q``, ``l<i>.mix.q.conv``, ``l<i>.mix.g``, ``l<i>.mlp.e<j>.gate``, ``l<i>.mlp.shared.sg``, ..., ``final.norm``, ``head``).

Notation: T tokens, W model width; H query heads over G key / value heads, key size d, value size e.
"""
from __future__ import annotations

import numpy as np


def f64(a):
    return np.asarray(a, np.float64)


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-f64(z)))


def silu(z):
    return z * sigmoid(z)


def linear(h, P, name):
    return f64(h) @ f64(P[name]).T


def tanh_norm(x, P, name):
    """No statistic of the row: every element by itself through tanh(alpha x), then weight and offset."""
    return np.tanh(float(np.asarray(P[name + ".alpha"]).reshape(())) * f64(x)) * f64(P[name]) + f64(P[name + ".b"])


def unit_rms(x, eps):
    """x / sqrt(mean(x^2) + eps) over the last axis."""
    x = f64(x)
    return x / np.sqrt((x * x).mean(-1, keepdims=True) + eps)


# ---- attention --------------------------------------------------------------------------------------------------------
def causal_conv(x, w):
    """x [T, C], w [C, taps] (last column: the current token), zeros before the start."""
    T, taps = x.shape[0], w.shape[1]
    xp = np.concatenate([np.zeros((taps - 1, x.shape[1])), f64(x)])
    return sum(xp[j:j + T] * f64(w)[:, j] for j in range(taps))


def frequencies(rot):
    """Angle per position of every pair.  Wavelengths above original / low are stretched by the factor, those below
    original / high are kept, in between the two frequencies are blended linearly in original / wavelength."""
    f = rot["base"] ** (-2.0 * np.arange(rot["dims"] // 2) / rot["dims"])
    sc = rot.get("scaling")
    if not sc:
        return f
    out = []
    for fi in f:
        wl = 2.0 * np.pi / fi
        if wl < sc["original"] / sc["high"]:
            out.append(fi)
        elif wl > sc["original"] / sc["low"]:
            out.append(fi / sc["factor"])
        else:
            t = (sc["original"] / wl - sc["low"]) / (sc["high"] - sc["low"])
            out.append((1.0 - t) * fi / sc["factor"] + t * fi)
    return np.array(out)


def rotate(x, rot):
    """x [T, heads, d]: the pairs (2i, 2i + 1) of the first dims elements turn by position * frequency i."""
    if not rot or not rot["dims"]:
        return f64(x)
    a = np.arange(x.shape[0])[:, None] * frequencies(rot)
    c, s = np.cos(a)[:, None], np.sin(a)[:, None]
    y = f64(x).copy()
    u, v = f64(x)[..., 0:rot["dims"]:2], f64(x)[..., 1:rot["dims"]:2]
    y[..., 0:rot["dims"]:2] = u * c - v * s
    y[..., 1:rot["dims"]:2] = v * c + u * s
    return y


def window_softmax_plus_one(score, window):
    """score [T, T], row i sees 0 <= i - j < window; 1 joins the denominator (a sink of score 0 without a value)."""
    T = score.shape[0]
    i, j = np.arange(T)[:, None], np.arange(T)[None, :]
    z = np.where((j <= i) & (i - j < window), score, -np.inf)
    m = np.maximum(z.max(-1, keepdims=True), 0.0)
    p = np.exp(z - m)
    return p / (p.sum(-1, keepdims=True) + np.exp(-m))


def queries_or_keys(h, P, name, n, mx, eps):
    """Projection, convolution, rotation, then every head over its own root mean square -> [T, n, d]."""
    x = causal_conv(linear(h, P, name), P[name + ".conv"]).reshape(h.shape[0], n, mx["dim"])
    return unit_rms(rotate(x, mx.get("rot")), eps)


def keys_and_values(h, P, pre, mx, eps):
    """What a layer caches: k [T, G, d] (convolved, rotated, normed) and v [T, G, e] (convolved)."""
    G = mx["kv_heads"]
    v = causal_conv(linear(h, P, pre + "v"), P[pre + "v.conv"]).reshape(h.shape[0], G, mx["vdim"])
    return queries_or_keys(h, P, pre + "k", G, mx, eps), v


def attention(h, P, pre, mx, eps, kv):
    """kv: the keys and values of this layer or of the one it borrows from; one sigmoid gate per head."""
    T = h.shape[0]
    H, G, e = mx["heads"], mx["kv_heads"], mx["vdim"]
    q = queries_or_keys(h, P, pre + "q", H, mx, eps)
    k, v = kv
    out = np.zeros((T, H, e))
    for hd in range(H):
        g = hd // (H // G)
        out[:, hd] = window_softmax_plus_one(q[:, hd] @ k[:, g].T * mx["scale"], mx["mask"]["size"]) @ v[:, g]
    out *= sigmoid(linear(h, P, pre + "g"))[:, :, None]
    return linear(out.reshape(T, H * e), P, pre + "o")


# ---- feed-forward -----------------------------------------------------------------------------------------------------
def gated_ff(h, P, pre):
    return linear(silu(linear(h, P, pre + "gate")) * linear(h, P, pre + "up"), P, pre + "down")


def route(h, P, pre, rt):
    """-> (indices [T, top], weights [T, top]): the largest logits, weights are the softmax over the chosen ones alone."""
    z = linear(h, P, pre + "router")
    sel = np.argsort(-z, -1, kind="stable")[:, :rt["top"]]
    zc = np.take_along_axis(z, sel, -1)
    w = np.exp(zc - zc.max(-1, keepdims=True))
    return sel, w / w.sum(-1, keepdims=True)


def mixture_ff(h, P, pre, ml):
    """The chosen experts' outputs times their weights, plus -- when there is one -- the expert of every token times a
    sigmoid of its own projection."""
    sel, wts = route(h, P, pre, ml["router"])
    out = np.zeros_like(f64(h))
    for j in range(ml["router"]["experts"]):
        at, slot = np.nonzero(sel == j)
        if len(at):
            out[at] += wts[at, slot][:, None] * gated_ff(h[at], P, f"{pre}e{j}.")
    if ml.get("shared"):
        out += sigmoid(linear(h, P, pre + "shared.sg")) * gated_ff(h, P, pre + "shared.")
    return out


# ---- the model --------------------------------------------------------------------------------------------------------
def forward(cfg, P, ids, return_layers=False):
    """Logits [T, vocab] of one sequence (and the residual stream after every layer)."""
    eps, mult = cfg["norm"]["eps"], cfg["residual_mult"]
    x = f64(P["embed"])[np.asarray(ids)] * cfg["embedding"]["scale"]
    layers, cached = [], []
    for li, ly in enumerate(cfg["layers"]):
        p, mx = f"l{li}.", ly["mixer"]
        h = tanh_norm(x, P, p + "norm1")
        j = mx.get("kv_from")
        cached.append(cached[j] if j is not None else keys_and_values(h, P, p + "mix.", mx, eps))
        x = x + mult * attention(h, P, p + "mix.", mx, eps, cached[li])
        if ly.get("mlp") is not None:
            x = x + mult * mixture_ff(tanh_norm(x, P, p + "norm2"), P, p + "mlp.", ly["mlp"])
        layers.append(x.copy())
    logits = linear(tanh_norm(x, P, "final.norm"), P, "head")
    return (logits, np.stack(layers)) if return_layers else logits


def greedy(cfg, P, prompt, n_new):
    ids = list(prompt)
    for _ in range(n_new):
        ids.append(int(np.argmax(forward(cfg, P, ids)[-1])))
    return ids[len(prompt):]
