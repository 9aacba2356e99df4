"""Test helpers for the Rirotar decoder: small configurations, random bfloat16-exact weights, checkpoints on disk."""
import numpy as np

from tests.korupel_util import bf16_round, tokens, write_checkpoint  # noqa: F401  (shared helpers, re-exported)


def latent(heads=3, dim=12, vdim=20, kv_rank=28, size=20, scale=None):
    return dict(heads=heads, dim=dim, vdim=vdim, kv_rank=kv_rank, scale=dim ** -0.5 if scale is None else scale, mask=dict(size=size))


def delta(heads=4, kv_heads=2, dim=12, vdim=20, conv=4):
    return dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, conv=conv)


def dense(ff=40, limit=1.5):
    return dict(kind="dense", ff=ff, limit=limit)


def moe(experts=6, top=2, ff=24, limit=1.0, groups=3, keep=2, scale=1.7):
    return dict(kind="moe", expert=dict(ff=ff, limit=limit), router=dict(experts=experts, top=top, groups=dict(count=groups, keep=keep), scale=scale))


def layer(kind, mixer, mlp):
    return dict(type=kind, mixer=mixer, mlp=mlp)


def config(layers, vocab=61, width=48, eps=2e-6, softcap=9.0):
    return dict(architecture="Rirotar", vocab=vocab, width=width, norm=dict(eps=eps), logit_softcap=softcap, layers=layers)


def small_config():
    """Every kind of mixer and feed-forward, a layer without one, sizes that are neither equal to each other nor powers of two."""
    return config([layer("channel_delta", delta(heads=3, kv_heads=3, dim=12, vdim=20, conv=4), moe(experts=6, top=2, ff=24, groups=3, keep=2)),
                   layer("latent_attention", latent(heads=3, dim=12, vdim=20, kv_rank=28, size=20), dense(ff=40)),
                   layer("delta", delta(heads=4, kv_heads=2, dim=20, vdim=12, conv=3), None),
                   layer("delta", delta(heads=2, kv_heads=1, dim=8, vdim=36, conv=5), moe(experts=8, top=3, ff=20, limit=0.7, groups=2, keep=1, scale=2.2)),
                   layer("latent_attention", latent(heads=2, dim=20, vdim=8, kv_rank=44, size=33, scale=0.3), dense(ff=28, limit=0.6)),
                   layer("channel_delta", delta(heads=4, kv_heads=2, dim=16, vdim=24, conv=2), dense(ff=36, limit=3.0))],
                  vocab=83, width=56)


def random_weights(cfg, seed=0, ranks=(6, 10)):
    """name -> float32 array (bfloat16-exact), in the checkpoint's spelling and shapes.  ranks: inner sizes of the two low-rank pairs."""
    rs = np.random.RandomState(seed)
    W, V = cfg["width"], cfg["vocab"]
    P = {}

    def mat(name, o, i, s=None):
        P[name] = bf16_round(rs.randn(o, i) * (s if s is not None else i ** -0.5))

    def vec(name, n, s=0.1, off=0.0):
        P[name] = bf16_round(off + s * rs.randn(n))

    mat("embed", V, W, 1.0)
    for li, ly in enumerate(cfg["layers"]):
        p, mx = f"l{li}.", ly["mixer"]
        q = p + "mix."
        vec(p + "norm1", W, 0.2)
        H, d, e = mx["heads"], mx["dim"], mx["vdim"]
        if ly["type"] == "latent_attention":
            r = mx["kv_rank"]
            mat(q + "q", H * d, W, 2.0 * W ** -0.5); mat(q + "dkv", r, W); vec(q + "dkv.norm", r, 0.2, 1.0)
            mat(q + "uk", H * d, r, 2.0 * r ** -0.5); mat(q + "uv", H * e, r)
            vec(q + "sink", H, 1.0, 0.5)
        else:
            G, taps = mx["kv_heads"], mx["conv"]
            for n, rows in (("q", G * d), ("k", G * d), ("v", H * e)):
                mat(q + n, rows, W)
                mat(q + n + ".conv", rows, taps, taps ** -0.5)
            mat(q + "b", H, W)
            vec(q + "A_log", H, 0.7, -0.5)
            vec(q + "norm", e, 0.2, 1.0)
            if ly["type"] == "delta":
                mat(q + "a", H, W); vec(q + "dt_bias", H, 0.5, -1.0); mat(q + "g", H * e, W)
            else:
                ar, gr = ranks
                mat(q + "a1", ar, W); mat(q + "a2", H * d, ar); vec(q + "dt_bias", H * d, 0.5, -1.0)
                mat(q + "g1", gr, W); mat(q + "g2", H * e, gr)
        mat(q + "o", W, H * e)
        ml = ly.get("mlp")
        if ml is None:
            continue
        vec(p + "norm2", W, 0.2)
        names = [p + "mlp."] if ml["kind"] == "dense" else [f"{p}mlp.e{x}." for x in range(ml["router"]["experts"])]
        ff = ml["ff"] if ml["kind"] == "dense" else ml["expert"]["ff"]
        for n in names:
            mat(n + "gate", ff, W, 2.0 * W ** -0.5); mat(n + "up", ff, W, 2.0 * W ** -0.5); mat(n + "down", W, ff)
        if ml["kind"] == "moe":
            mat(p + "mlp.router", ml["router"]["experts"], W, 2.0 * W ** -0.5)
    vec("final.norm", W, 0.2)
    mat("head", V, W, 2.0 * W ** -0.5)
    return P


def planted_window(size, heads=2, dim=8, vdim=8, kv_rank=16, alpha=6.0):
    """One latent-attention layer in which a query token QT sees a key token KT stand out among whatever else is visible: embedding
    coordinate 0 is set for KT only and feeds latent element 0 alone, coordinate 1 is set for QT only and feeds query element 0, which
    the key up-projection ties to latent element 0."""
    cfg = config([layer("latent_attention", latent(heads=heads, dim=dim, vdim=vdim, kv_rank=kv_rank, size=size, scale=1.0), None)], vocab=67, width=40,
                 softcap=50.0)
    P = random_weights(cfg, 7)
    QT, KT = 65, 66
    P["embed"][:, :2] = 0
    P["embed"][KT, 0] = 4.0
    P["embed"][QT, 1] = 4.0
    P["l0.norm1"][:] = 0
    q = "l0.mix."
    P[q + "q"] = bf16_round(P[q + "q"] * 0.1)
    P[q + "dkv"][:, :2] = 0
    P[q + "dkv"][0] = 0
    P[q + "dkv"][0, 0] = alpha
    P[q + "dkv.norm"][:] = 1.0
    for h in range(heads):
        P[q + "q"][h * dim] = 0
        P[q + "q"][h * dim, 1] = alpha
        P[q + "uk"][h * dim] = 0
        P[q + "uk"][h * dim, 0] = 1.0
    return cfg, P, QT, KT


def slow_decay(kind):
    """One delta-rule layer whose decays and write strengths leave a token's trace for hundreds of steps."""
    cfg = config([layer(kind, delta(heads=2, kv_heads=1, dim=16, vdim=8, conv=2), None)], vocab=37, width=24)
    P = random_weights(cfg, 9)
    P["l0.mix.A_log"][:] = -7.0
    P["l0.mix.b"] = bf16_round(P["l0.mix.b"] * 0.1)
    P["l0.mix.b"][:, 0] = -3.0
    P["embed"][:, 0] = 1.5                                        # write strengths around sigmoid(-4)
    return cfg, P
