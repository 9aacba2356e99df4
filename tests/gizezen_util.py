"""Test helpers for the Gizezen decoder: small configurations, random bfloat16-exact weights, checkpoints on disk."""
import numpy as np

from tests.korupel_util import bf16_round, tokens, write_checkpoint  # noqa: F401  (shared helpers, re-exported)


def bands(factor=3.0, low=1.0, high=4.0, original=60):
    return dict(factor=factor, low=low, high=high, original=original)


def attn(heads=4, kv_heads=2, dim=12, vdim=20, conv=3, size=20, scale=None, rot_dims=8, base=700.0, scaling=None, kv_from=None):
    mx = dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, conv=conv, scale=dim ** -0.5 if scale is None else scale, mask=dict(size=size),
              rot=dict(base=base, dims=rot_dims))
    if scaling:
        mx["rot"]["scaling"] = scaling
    if kv_from is not None:
        mx["kv_from"] = kv_from
    return mx


def moe(experts=6, top=2, ff=24, shared=28):
    ml = dict(kind="moe", expert=dict(ff=ff), router=dict(experts=experts, top=top))
    if shared:
        ml["shared"] = dict(ff=shared)
    return ml


def layer(mixer, mlp):
    return dict(type="attention", mixer=mixer, mlp=mlp)


def config(layers, vocab=61, width=48, eps=3e-6, mult=0.4, embed_scale=2.5):
    return dict(architecture="Gizezen", vocab=vocab, width=width, norm=dict(eps=eps), embedding=dict(scale=embed_scale), residual_mult=mult,
                layers=layers)


def small_config():
    """Keys of their own and borrowed ones (twice from the same layer, across another), different windows, taps and rotations on the two
    sides of a loan, with and without feed-forward and shared expert; sizes that are neither equal to each other nor powers of two."""
    return config([layer(attn(heads=4, kv_heads=2, dim=12, vdim=20, conv=3, size=20, rot_dims=8, scaling=bands()), moe(experts=6, top=2, ff=24, shared=28)),
                   layer(attn(heads=6, kv_heads=2, dim=12, vdim=20, conv=4, size=33, rot_dims=12, base=90.0, scale=0.5, kv_from=0), None),
                   layer(attn(heads=3, kv_heads=3, dim=20, vdim=12, conv=5, size=15, rot_dims=20, scaling=bands(2.0, 0.5, 3.0, 40)), moe(experts=9, top=3, ff=20, shared=0)),
                   layer(attn(heads=2, kv_heads=2, dim=12, vdim=20, conv=2, size=20, rot_dims=4, kv_from=0), moe(experts=5, top=1, ff=36, shared=12)),
                   layer(attn(heads=2, kv_heads=1, dim=28, vdim=36, conv=1, size=70, rot_dims=0, scale=0.3), moe(experts=4, top=4, ff=16, shared=20))],
                  vocab=83, width=56)


def random_weights(cfg, seed=0):
    """name -> float32 array (bfloat16-exact), in the checkpoint's spelling and shapes."""
    rs = np.random.RandomState(seed)
    W, V = cfg["width"], cfg["vocab"]
    P = {}

    def mat(name, o, i, s=None):
        P[name] = bf16_round(rs.randn(o, i) * (s if s is not None else i ** -0.5))

    def norm(name):
        P[name] = bf16_round(1.0 + 0.2 * rs.randn(W))
        P[name + ".b"] = bf16_round(0.2 * rs.randn(W))
        P[name + ".alpha"] = bf16_round(np.array(0.3 + 0.5 * rs.rand())).reshape(())          # a scalar tensor

    mat("embed", V, W, 0.5)
    for li, ly in enumerate(cfg["layers"]):
        p, mx = f"l{li}.", ly["mixer"]
        q = p + "mix."
        norm(p + "norm1")
        H, G, d, e, taps = mx["heads"], mx["kv_heads"], mx["dim"], mx["vdim"], mx["conv"]
        for n, rows in (("q", H * d), ("k", G * d), ("v", G * e)):
            if n != "q" and mx.get("kv_from") is not None:
                continue
            mat(q + n, rows, W)
            mat(q + n + ".conv", rows, taps, taps ** -0.5)
        mat(q + "g", H, W, 2.0 * W ** -0.5)
        mat(q + "o", W, H * e, 2.0 * (H * e) ** -0.5)
        ml = ly.get("mlp")
        if ml is None:
            continue
        norm(p + "norm2")
        experts = [(f"{p}mlp.e{x}.", ml["expert"]["ff"]) for x in range(ml["router"]["experts"])]
        if ml.get("shared"):
            experts.append((p + "mlp.shared.", ml["shared"]["ff"]))
            mat(p + "mlp.shared.sg", 1, W, 2.0 * W ** -0.5)
        for n, ff in experts:
            mat(n + "gate", ff, W, 2.0 * W ** -0.5); mat(n + "up", ff, W, 2.0 * W ** -0.5); mat(n + "down", W, ff)
        mat(p + "mlp.router", ml["router"]["experts"], W, 2.0 * W ** -0.5)
    norm("final.norm")
    mat("head", V, W, 2.0 * W ** -0.5)
    return P


def planted_window(size, borrowed_size=None, heads=2, kv_heads=1, dim=16, vdim=8, width=40):
    """A layer in which a query token QT sees a key token KT stand out among whatever else is visible: coordinate 0 of the normed input is
    set for KT alone and feeds one key element (which nothing else feeds, and which does not rotate), coordinate 1 is set for QT alone and
    feeds the same element of every query; KT's value is large.  borrowed_size: a second layer with a window of that size on the first
    one's keys, and the first layer's own output switched off.  The convolutions pass the current token only."""
    layers = [layer(attn(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, conv=3, size=size, scale=1.0, rot_dims=dim - 4), None)]
    if borrowed_size is not None:
        layers.append(layer(attn(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, conv=2, size=borrowed_size, scale=1.0, rot_dims=dim - 4, kv_from=0), None))
    cfg = config(layers, vocab=67, width=width, mult=1.0, embed_scale=1.0)
    P = random_weights(cfg, 7)
    QT, KT, last = 65, 66, dim - 1
    P["embed"][:, :2] = 0
    P["embed"][KT, 0] = 4.0
    P["embed"][QT, 1] = 4.0
    for li, ly in enumerate(cfg["layers"]):
        q = f"l{li}.mix."
        P[f"l{li}.norm1.b"][:2] = 0
        for n in "qkv":
            if q + n not in P:
                continue
            P[q + n + ".conv"][:] = 0
            P[q + n + ".conv"][:, -1] = 1.0
        P[q + "q"][:, :2] = 0
        for h in range(heads):
            P[q + "q"][h * dim + last] = 0
            P[q + "q"][h * dim + last, 1] = 24.0
        P[q + "o"] = bf16_round(P[q + "o"] * 2.0)
        P[q + "o"][:2] = 0                                        # (coordinates 0 and 1 stay what the embedding says)
        if q + "k" in P:
            P[q + "k"][:, :2] = 0
            P[q + "v"][:, 0] = 3.0
            for g in range(kv_heads):
                P[q + "k"][g * dim + last] = 0
                P[q + "k"][g * dim + last, 0] = 24.0
    if borrowed_size is not None:
        P["l0.mix.o"][:] = 0
    return cfg, P, QT, KT
