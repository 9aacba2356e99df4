"""Plain NumPy statement of the Rirotar decoder, one function per mechanism (float64, whole sequences, no cache).

Test infrastructure only: nothing here is imported by the product.  A model is a config dict in the checkpoint's own
spelling (``architecture``, ``width``, ``vocab``, ``norm.eps``, ``logit_softcap``, ``layers[...]``) and a dict of arrays under
the checkpoint's tensor names (``embed``, ``l<i>.norm1``, ``l<i>.mix.q``, ``l<i>.mix.q.conv``, ``l<i>.mix.dkv.norm``,
``l<i>.mlp.e<j>.gate``, ..., ``final.norm``, ``head``).

Notation: T tokens, W model width.  Latent attention: H heads of d query / key and e value elements, latent size r.  Delta
recurrences: H heads of d key and e value elements over G query / key heads, state [d][e].
"""
from __future__ import annotations

import numpy as np


def f64(a):
    return np.asarray(a, np.float64)


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-f64(z)))


def silu(z):
    return z * sigmoid(z)


def softplus(z):
    z = f64(z)
    return np.maximum(z, 0.0) + np.log1p(np.exp(-np.abs(z)))


def unit_rms(x, eps):
    """x / sqrt(mean(x^2) + eps) over the last axis."""
    x = f64(x)
    return x / np.sqrt((x * x).mean(-1, keepdims=True) + eps)


def unit_length(x):
    """x / sqrt(sum(x^2) + 1e-6) over the last axis."""
    x = f64(x)
    return x / np.sqrt((x * x).sum(-1, keepdims=True) + 1e-6)


def layer_norm1p(x, w, eps):
    """RMS norm whose weight is stored around zero."""
    return unit_rms(x, eps) * (1.0 + f64(w))


def linear(h, P, name):
    return f64(h) @ f64(P[name]).T


# ---- latent attention -------------------------------------------------------------------------------------------------
def window_softmax_with_sink(score, sink, window):
    """score [T, T], row i sees 0 <= i - j < window; exp(sink) joins the denominator once."""
    T = score.shape[0]
    i, j = np.arange(T)[:, None], np.arange(T)[None, :]
    z = np.where((j <= i) & (i - j < window), score, -np.inf)
    m = np.maximum(z.max(-1, keepdims=True), sink)
    p = np.exp(z - m)
    return p / (p.sum(-1, keepdims=True) + np.exp(sink - m))


def latent_attention(h, P, pre, mx, eps):
    """Keys and values are up-projections of one normed latent per token; sliding window, a sink per head, no positions."""
    T = h.shape[0]
    H, d, e = mx["heads"], mx["dim"], mx["vdim"]
    q = linear(h, P, pre + "q").reshape(T, H, d)
    c = unit_rms(linear(h, P, pre + "dkv"), eps) * f64(P[pre + "dkv.norm"])
    k = linear(c, P, pre + "uk").reshape(T, H, d)
    v = linear(c, P, pre + "uv").reshape(T, H, e)
    out = np.zeros((T, H, e))
    for hd in range(H):
        w = window_softmax_with_sink(q[:, hd] @ k[:, hd].T * mx["scale"], float(P[pre + "sink"][hd]), mx["mask"]["size"])
        out[:, hd] = w @ v[:, hd]
    return linear(out.reshape(T, H * e), P, pre + "o")


# ---- delta recurrences ------------------------------------------------------------------------------------------------
def causal_conv(x, w):
    """x [T, C], w [C, taps] (last column: the current token), zeros before the start."""
    T, taps = x.shape[0], w.shape[1]
    xp = np.concatenate([np.zeros((taps - 1, x.shape[1])), f64(x)])
    return sum(xp[j:j + T] * f64(w)[:, j] for j in range(taps))


def delta_inputs(h, P, pre, mx):
    """Convolved, activated and normed q [T, G, d], k [T, G, d], v [T, H, e] and the write strength beta [T, H]."""
    T = h.shape[0]
    H, G, d, e = mx["heads"], mx["kv_heads"], mx["dim"], mx["vdim"]
    q, k, v = (silu(causal_conv(linear(h, P, pre + n), P[pre + n + ".conv"])) for n in "qkv")
    q = unit_length(q.reshape(T, G, d)) * d ** -0.5
    k = unit_length(k.reshape(T, G, d))
    return q, k, v.reshape(T, H, e), sigmoid(linear(h, P, pre + "b"))


def head_log_decay(h, P, pre, mx):
    """[T, H]: the logarithm of one decay per head."""
    return -np.exp(f64(P[pre + "A_log"])) * softplus(linear(h, P, pre + "a") + f64(P[pre + "dt_bias"]))


def channel_log_decay(h, P, pre, mx):
    """[T, H, d]: the logarithm of one decay per head and key channel, from a low-rank pair."""
    T, H, d = h.shape[0], mx["heads"], mx["dim"]
    z = softplus(linear(linear(h, P, pre + "a1"), P, pre + "a2") + f64(P[pre + "dt_bias"])).reshape(T, H, d)
    return -np.exp(f64(P[pre + "A_log"]))[:, None] * z


def delta_rule(q, k, v, beta, log_decay):
    """S <- g S; u = beta (v - S^T k); S <- S + k u^T; o = S^T q.  log_decay [T, H] or [T, H, d] -> o [T, H, e]."""
    T, G, d = q.shape
    H, e = v.shape[1:]
    g = np.exp(log_decay if log_decay.ndim == 3 else log_decay[:, :, None])
    S = np.zeros((H, d, e))
    o = np.zeros((T, H, e))
    for t in range(T):
        for hd in range(H):
            kt, qt = k[t, hd // (H // G)], q[t, hd // (H // G)]
            S[hd] = g[t, hd][:, None] * S[hd]
            u = beta[t, hd] * (v[t, hd] - S[hd].T @ kt)
            S[hd] += np.outer(kt, u)
            o[t, hd] = S[hd].T @ qt
    return o


def gated_output(o, gate, P, pre, eps):
    """Unit RMS per head, one weight vector for all heads, gate [T, H e], output projection."""
    T = o.shape[0]
    y = (unit_rms(o, eps) * f64(P[pre + "norm"])).reshape(T, -1)
    return linear(y * gate, P, pre + "o")


def delta(h, P, pre, mx, eps):
    q, k, v, beta = delta_inputs(h, P, pre, mx)
    o = delta_rule(q, k, v, beta, head_log_decay(h, P, pre, mx))
    return gated_output(o, silu(linear(h, P, pre + "g")), P, pre, eps)


def channel_delta(h, P, pre, mx, eps):
    q, k, v, beta = delta_inputs(h, P, pre, mx)
    o = delta_rule(q, k, v, beta, channel_log_decay(h, P, pre, mx))
    return gated_output(o, sigmoid(linear(linear(h, P, pre + "g1"), P, pre + "g2")), P, pre, eps)


# ---- feed-forward -----------------------------------------------------------------------------------------------------
def capped_ff(h, P, pre, limit):
    """g = min(W_gate h, limit), u = clamp(W_up h, +-limit): W_down (g sigmoid(1.702 g) (u + 1))."""
    g = np.minimum(linear(h, P, pre + "gate"), limit)
    u = np.clip(linear(h, P, pre + "up"), -limit, limit)
    return linear(g * sigmoid(1.702 * g) * (u + 1.0), P, pre + "down")


def route(h, P, pre, rt):
    """-> (indices [T, top], weights [T, top]).  Sigmoid scores; only experts of the best groups (the sum of a group's two
    largest scores) can be chosen; weights divided by their sum, times the scale."""
    s = sigmoid(linear(h, P, pre + "router"))
    T, E = s.shape
    gc, keep = rt["groups"]["count"], rt["groups"]["keep"]
    parts = s.reshape(T, gc, E // gc)
    group_score = np.sort(parts, -1)[:, :, -2:].sum(-1)
    kept = np.argsort(-group_score, -1, kind="stable")[:, :keep]
    allowed = np.zeros((T, gc), bool)
    np.put_along_axis(allowed, kept, True, -1)
    masked = np.where(np.repeat(allowed, E // gc, -1), s, -np.inf)
    sel = np.argsort(-masked, -1, kind="stable")[:, :rt["top"]]
    w = np.take_along_axis(s, sel, -1)
    return sel, w / (w.sum(-1, keepdims=True) + 1e-20) * rt["scale"]


def mixture_ff(h, P, pre, ml):
    sel, wts = route(h, P, pre, ml["router"])
    out = np.zeros_like(f64(h))
    for t in range(h.shape[0]):
        for j, w in zip(sel[t], wts[t]):
            out[t] += w * capped_ff(f64(h[t:t + 1]), P, f"{pre}e{j}.", ml["expert"]["limit"])[0]
    return out


# ---- the model --------------------------------------------------------------------------------------------------------
MIXERS = {"latent_attention": latent_attention, "delta": delta, "channel_delta": channel_delta}


def forward(cfg, P, ids, return_layers=False):
    """Logits [T, vocab] of one sequence (and the residual stream after every layer)."""
    eps = cfg["norm"]["eps"]
    x = f64(P["embed"])[np.asarray(ids)]
    layers = []
    for li, ly in enumerate(cfg["layers"]):
        p = f"l{li}."
        x = x + MIXERS[ly["type"]](layer_norm1p(x, P[p + "norm1"], eps), P, p + "mix.", ly["mixer"], eps)
        ml = ly.get("mlp")
        if ml is not None:
            h = layer_norm1p(x, P[p + "norm2"], eps)
            x = x + (capped_ff(h, P, p + "mlp.", ml["limit"]) if ml["kind"] == "dense" else mixture_ff(h, P, p + "mlp.", ml))
        layers.append(x.copy())
    logits = linear(layer_norm1p(x, P["final.norm"], eps), P, "head")
    cap = cfg["logit_softcap"]
    logits = cap * np.tanh(logits / cap)
    return (logits, np.stack(layers)) if return_layers else logits


def greedy(cfg, P, prompt, n_new):
    ids = list(prompt)
    for _ in range(n_new):
        ids.append(int(np.argmax(forward(cfg, P, ids)[-1])))
    return ids[len(prompt):]
