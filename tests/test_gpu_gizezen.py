"""GPU: the Gizezen decoder in the library (kernels_layered.hip, kernels_layered_mix.hip, model_layered.cpp, the engine's mixed
steps) against the plain NumPy statement oracle/gizezen_oracle.py, on small configurations with random weights made here.

float32 compute is the sharp comparison (TOL_F32 relative to the largest logit); bfloat16 compute is checked against the
same oracle with the rounding's own allowance, and against itself across schedules."""
import numpy as np
import pytest

from oracle import gizezen_oracle as O
from tests import gizezen_util as U

pytestmark = pytest.mark.gpu

TOL_F32 = 1e-4
TOL_BF16 = 6e-2


def _load(tmp_path, cfg, P, dtype="float32", **kw):
    from crane_amd.backend import Model
    kw.setdefault("max_seq_len", 512)
    kw.setdefault("max_seqs", 4)
    return Model.from_pretrained(U.write_checkpoint(str(tmp_path / "ckpt"), cfg, P), compute_dtype=dtype, **kw)


def _err(got, want):
    want = np.asarray(want, np.float64)
    return float(np.abs(np.asarray(got, np.float64) - want).max() / np.abs(want).max())


def _err_most(got, want):
    """bfloat16 format: the error that nine positions in ten stay under.  A router's close call that the rounding decides the other
    way moves one position by a whole expert; no test rests on those."""
    want = np.asarray(want, np.float64)
    per = np.abs(np.asarray(got, np.float64) - want).max(-1) / np.abs(want).max()
    assert np.median(per) < 0.03, float(np.median(per))
    return float(np.quantile(per, 0.9))


def _all(n):
    return list(range(n))


def _one(mixer, mlp=None, **kw):
    return U.config([U.layer(mixer, mlp)], **kw)


SINGLE = {
    "attention": _one(U.attn()),
    "attention, a key head per query head, one tap, window of one": _one(U.attn(heads=3, kv_heads=3, dim=8, vdim=12, conv=1, size=1, rot_dims=8)),
    "attention, one key head, odd sizes, two taps, nothing rotates": _one(U.attn(heads=5, kv_heads=1, dim=7, vdim=9, conv=2, rot_dims=0)),
    "attention, seven taps, window of a page": _one(U.attn(heads=2, kv_heads=1, dim=16, vdim=16, conv=7, size=64, rot_dims=16)),
    "attention, odd value size, a part of the head rotates": _one(U.attn(heads=4, kv_heads=2, dim=14, vdim=5, conv=4, rot_dims=6, scale=0.6)),
    "banded frequencies": _one(U.attn(dim=16, rot_dims=16, base=3000.0, size=90, scaling=U.bands(5.0, 1.0, 4.0, 80))),
    "banded frequencies, wide band": _one(U.attn(dim=16, rot_dims=12, base=500.0, size=90, scaling=U.bands(8.0, 0.25, 16.0, 64))),
    "borrowed keys and values": U.config([U.layer(U.attn(), None), U.layer(U.attn(heads=2, conv=4, size=31, rot_dims=12, kv_from=0), None)]),
    "keys lent over a layer with its own, twice": U.config([U.layer(U.attn(), None), U.layer(U.attn(heads=3, kv_heads=1, dim=20, vdim=8, conv=2), None),
                                                            U.layer(U.attn(heads=6, kv_heads=2, conv=2, kv_from=0), None),
                                                            U.layer(U.attn(heads=1, kv_heads=1, dim=20, vdim=8, conv=3, kv_from=1), None),
                                                            U.layer(U.attn(size=7, kv_from=0), None)]),
    "experts": _one(U.attn(), U.moe(shared=0)),
    "experts and a shared one": _one(U.attn(), U.moe()),
    "all experts chosen": _one(U.attn(), U.moe(experts=5, top=5, shared=0)),
    "one expert of one, and a shared one": _one(U.attn(), U.moe(experts=1, top=1, ff=20, shared=44)),
    "a residual multiplier above one": _one(U.attn(), U.moe(), mult=1.7, embed_scale=0.3),
}


@pytest.mark.parametrize("name", list(SINGLE))
def test_each_mechanism_alone_whole_prompt_and_layer_rows(tmp_path, name):
    cfg = SINGLE[name]
    P = U.random_weights(cfg, 1)
    toks = U.tokens(101, cfg["vocab"], 1)
    want, layers = O.forward(cfg, P, toks, True)
    m = _load(tmp_path, cfg, P)
    try:
        m.layer_capture(True)
        s = m.seq_alloc()
        got, greedy = m.step_batch([(s, toks, _all(len(toks)))])
        rows = m.layer_rows().reshape(len(cfg["layers"]), len(toks), cfg["width"])
        assert _err(rows, layers) < TOL_F32
        assert _err(got, want) < TOL_F32
        assert list(greedy) == [int(np.argmax(r)) for r in got]
    finally:
        m.close()


def test_prefill_against_token_by_token_decoding(tmp_path):
    cfg = U.small_config()
    P = U.random_weights(cfg, 2)
    toks = U.tokens(80, cfg["vocab"], 2)
    want = O.forward(cfg, P, toks)
    m = _load(tmp_path, cfg, P)
    try:
        a, b = m.seq_alloc(), m.seq_alloc()
        whole, _ = m.step_batch([(a, toks, _all(len(toks)))])
        serial = np.concatenate([m.step_batch([(b, [t], [0])])[0] for t in toks])
        assert _err(whole, want) < TOL_F32 and _err(serial, want) < TOL_F32
        assert _err(serial, whole) < TOL_F32
    finally:
        m.close()


@pytest.mark.parametrize("cuts", [[2] * 12 + [3, 5, 2, 7, 1, 1, 2, 16, 2], [64, 2, 1, 3], [1, 69], [33, 33, 4], [5, 60, 2, 2, 1], [17, 16, 65, 64, 15], [129, 3]])
def test_portions_of_several_sizes_down_to_two_tokens(tmp_path, cuts):
    cfg = U.small_config()
    P = U.random_weights(cfg, 3)
    n = sum(cuts)
    toks = U.tokens(n, cfg["vocab"], 3)
    want = O.forward(cfg, P, toks)
    m = _load(tmp_path, cfg, P)
    try:
        s, at, out = m.seq_alloc(), 0, []
        for c in cuts:
            out.append(m.step_batch([(s, toks[at:at + c], _all(c))])[0])
            at += c
        assert m.seq_len(s) == n
        assert _err(np.concatenate(out), want) < TOL_F32
    finally:
        m.close()


def test_batches_of_unequal_requests_against_each_alone(tmp_path):
    cfg = U.small_config()
    P = U.random_weights(cfg, 4)
    reqs = [U.tokens(n, cfg["vocab"], 10 + i) for i, n in enumerate((67, 5, 130, 31))]
    want = [O.forward(cfg, P, t) for t in reqs]
    # per step: (request, tokens taken) -- long portions beside single decode tokens, requests joining and pausing
    plan = [[(0, 40), (1, 2)], [(0, 1), (1, 1), (2, 64)], [(2, 2), (0, 1), (3, 30)], [(1, 2), (2, 60), (3, 1), (0, 25)], [(2, 0)]]
    m = _load(tmp_path, cfg, P)
    try:
        seqs = [m.seq_alloc() for _ in reqs]
        at = [0] * len(reqs)
        got = [[] for _ in reqs]
        for step in plan:
            step = [(r, c if c else len(reqs[r]) - at[r]) for r, c in step]
            out, _ = m.step_batch([(seqs[r], reqs[r][at[r]:at[r] + c], _all(c)) for r, c in step])
            row = 0
            for r, c in step:
                got[r].append(out[row:row + c])
                row += c
                at[r] += c
        for r in range(len(reqs)):
            have = np.concatenate(got[r])
            assert _err(have, want[r][:len(have)]) < TOL_F32, r
        assert at[2] == 130 and at[0] == 67
    finally:
        m.close()


def test_pages_and_slots_that_are_freed_and_used_again(tmp_path):
    cfg = U.small_config()
    P = U.random_weights(cfg, 5)
    m = _load(tmp_path, cfg, P, max_seq_len=192, kv_pool_tokens=256, max_seqs=2)        # 4 pages of 64, 2 slots
    try:
        for rnd in range(3):
            reqs = [U.tokens(n, cfg["vocab"], 20 + 2 * rnd + i) for i, n in enumerate((100 + 7 * rnd, 90 - 11 * rnd))]
            seqs = [m.seq_alloc(), m.seq_alloc()]
            with pytest.raises(Exception):
                m.seq_alloc()                                     # both slots taken
            out, _ = m.step_batch([(seqs[0], reqs[0][:50], []), (seqs[1], reqs[1], _all(len(reqs[1])))])
            assert _err(out, O.forward(cfg, P, reqs[1])) < TOL_F32
            out, _ = m.step_batch([(seqs[0], reqs[0][50:], _all(len(reqs[0]) - 50))])
            assert _err(out, O.forward(cfg, P, reqs[0])[50:]) < TOL_F32
            assert m.active_kv_cache_bytes() > 0
            for s in seqs:
                m.seq_free(s)
            assert m.active_kv_cache_bytes() == 0
        # a step that does not fit in the pool fails and leaves the sequence as it was
        a, b = m.seq_alloc(), m.seq_alloc()
        m.step_batch([(a, U.tokens(150, cfg["vocab"], 1), None)])
        with pytest.raises(Exception):
            m.step_batch([(b, U.tokens(120, cfg["vocab"], 2), None)])
        assert m.seq_len(b) == 0 and m.seq_len(a) == 150
    finally:
        m.close()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("decoded", [False, True])
@pytest.mark.parametrize("size,borrowed", [(20, None), (64, None), (5, None), (20, 33), (64, 7)])
def test_planted_keys_at_the_edges_of_the_window_and_at_page_borders(tmp_path, dtype, decoded, size, borrowed):
    cfg, P, QT, KT = U.planted_window(size, borrowed)             # borrowed: a second layer with a window of its own on the first one's keys
    size = borrowed or size
    tol = TOL_F32 if dtype == "float32" else 3e-2
    m = _load(tmp_path, cfg, P, dtype=dtype)
    try:
        # (key position, query position): the window's last and first-outside position, keys on both sides of a page border (pages
        # of 64 tokens), the same far into the sequence
        cases = [(0, size - 1), (0, size), (1, size), (63, 64), (64, 65), (63, 63 + size - 1), (63, 63 + size), (64, 64 + size - 1), (64, 64 + size),
                 (3, 199), (199 - size + 1, 199), (199 - size, 199), (127, 128), (128, 128 + size - 1), (128, 128 + size)]
        for kp, qp in cases:
            if not 0 <= kp < qp < 200:
                continue
            toks = U.tokens(200, 65, kp * 1000 + qp)
            toks[kp], toks[qp] = KT, QT
            want = O.forward(cfg, P, toks[:qp + 1])
            plain = list(toks)
            plain[kp] = (toks[kp - 1] + 1) % 65 if kp else 1
            moved = float(np.abs(O.forward(cfg, P, plain[:qp + 1])[qp] - want[qp]).max() / np.abs(want[qp]).max())
            seen = qp - kp < size
            assert (moved > 0.1) == seen and (seen or moved < 1e-3), (kp, qp, moved)       # the planted key matters exactly where the mask shows it
            s = m.seq_alloc()
            if decoded:
                lo = max(1, qp - 2)
                m.step_batch([(s, toks[:lo], [])])
                got = np.concatenate([m.step_batch([(s, [toks[p]], [0])])[0] for p in range(lo, qp + 1)])
                assert _err(got, want[lo:qp + 1]) < tol, (kp, qp)
            else:
                got, _ = m.step_batch([(s, toks[:qp + 1], [qp - 1, qp])])
                assert _err(got, want[qp - 1:qp + 1]) < tol, (kp, qp)
            m.seq_free(s)
    finally:
        m.close()


def _far_below_zero(heads=2, kv_heads=1, dim=8, score=-5.5, size=300):
    """Every score is the same number far below zero: the window's keys together weigh about as much as the one in the denominator."""
    cfg = _one(U.attn(heads=heads, kv_heads=kv_heads, dim=dim, vdim=16, conv=2, size=size, scale=-score / dim, rot_dims=0))
    P = U.random_weights(cfg, 21)
    P["l0.norm1"][0], P["l0.norm1.b"][0] = 0.0, 1.0
    for n, rows, sign in (("q", heads, 1.0), ("k", kv_heads, -1.0)):
        P["l0.mix." + n][:] = 0
        P["l0.mix." + n][:, 0] = sign * 4.0
        P["l0.mix." + n + ".conv"][:] = [0.0, 1.0]
    P["l0.mix.v"] = U.bf16_round(P["l0.mix.v"] * 4.0)
    P["l0.mix.v"][:, 0] = 3.0
    return cfg, P


def test_the_one_in_the_denominator_counts_once_in_prompts_and_with_split_keys(tmp_path, monkeypatch):
    cfg, P = _far_below_zero()
    toks = U.tokens(400, cfg["vocab"], 21)
    want = O.forward(cfg, P, toks)
    with monkeypatch.context() as mp:                             # left out or taken twice it shows
        plus = O.window_softmax_plus_one
        mp.setattr(O, "window_softmax_plus_one", lambda s, w: (lambda p: p / p.sum(-1, keepdims=True))(plus(s, w)))
        assert _err(O.forward(cfg, P, toks), want) > 0.05
        mp.setattr(O, "window_softmax_plus_one", lambda s, w: (lambda p: p / (2.0 - p.sum(-1, keepdims=True)))(plus(s, w)))
        assert _err(O.forward(cfg, P, toks), want) > 0.05
    for dtype, tol in (("float32", TOL_F32), ("bfloat16", 3e-2)):
        m = _load(tmp_path, cfg, P, dtype=dtype)
        try:
            a, b = m.seq_alloc(), m.seq_alloc()
            assert _err(m.step_batch([(a, toks, _all(400))])[0], want) < tol
            m.step_batch([(b, toks[:380], [])])
            assert _err(np.concatenate([m.step_batch([(b, [t], [0])])[0] for t in toks[380:]]), want[380:]) < tol
        finally:
            m.close()


def test_scores_far_above_and_far_below_zero(tmp_path):
    """Unit heads times a large scale: exponentials of some hundred on both sides of the sink's zero."""
    cfg = U.config([U.layer(U.attn(heads=3, kv_heads=1, dim=12, vdim=8, scale=30.0, rot_dims=4), None)])
    P = U.random_weights(cfg, 22)
    toks = U.tokens(120, cfg["vocab"], 22)
    want = O.forward(cfg, P, toks)
    m = _load(tmp_path, cfg, P)
    try:
        a, b = m.seq_alloc(), m.seq_alloc()
        got, _ = m.step_batch([(a, toks, _all(120))])
        assert np.isfinite(got).all() and _err(got, want) < 10 * TOL_F32       # (a score of 300 has lost two digits)
        assert _err(np.concatenate([m.step_batch([(b, toks[at:at + 8], _all(8))])[0] for at in range(0, 120, 8)]), want) < 10 * TOL_F32
    finally:
        m.close()


def test_convolution_tails_over_every_cut_of_a_portion(tmp_path):
    """Six taps: an impulse in the input shows in the next five tokens' queries, keys and values wherever the portions are cut."""
    cfg = U.config([U.layer(U.attn(conv=6, size=40), None), U.layer(U.attn(conv=5, size=40, kv_from=0), None)])
    P = U.random_weights(cfg, 23)
    for n in "qkv":
        P["l0.mix." + n + ".conv"] = U.bf16_round(P["l0.mix." + n + ".conv"] * 3.0)
    toks = U.tokens(24, cfg["vocab"], 23)
    want = O.forward(cfg, P, toks)
    m = _load(tmp_path, cfg, P)
    try:
        for cut in range(1, 23):
            for second in (1, 2, 3, 24):
                s, out, at = m.seq_alloc(), [], 0
                for c in (cut, second, 24):
                    c = min(c, 24 - at)
                    if c:
                        out.append(m.step_batch([(s, toks[at:at + c], _all(c))])[0])
                        at += c
                assert _err(np.concatenate(out), want) < TOL_F32, (cut, second)
                m.seq_free(s)
    finally:
        m.close()


def test_far_positions_turn_by_their_own_angle(tmp_path):
    """A high base and a window of hundreds: a rotation that restarts with the portion or the page would show."""
    cfg = _one(U.attn(heads=2, kv_heads=1, dim=16, vdim=8, size=400, rot_dims=16, base=5e4, scale=1.5, scaling=U.bands(4.0, 1.0, 4.0, 512)))
    P = U.random_weights(cfg, 24)
    toks = U.tokens(500, cfg["vocab"], 24)
    want = O.forward(cfg, P, toks)
    plain = dict(cfg, layers=[U.layer(dict(cfg["layers"][0]["mixer"], rot=dict(base=5e4, dims=16)), None)])
    assert _err(O.forward(plain, P, toks)[300:], want[300:]) > 0.02           # the stretched frequencies matter
    m = _load(tmp_path, cfg, P)
    try:
        s, at, out = m.seq_alloc(), 0, []
        for c in [130, 2, 68, 200] + [1] * 40 + [60]:
            out.append(m.step_batch([(s, toks[at:at + c], _all(c))])[0])
            at += c
        assert at == 500 and _err(np.concatenate(out), want) < 3 * TOL_F32     # (angles of hundreds of radians in 32 bits)
    finally:
        m.close()


def test_first_tokens_of_a_sequence(tmp_path):
    cfg = U.small_config()
    P = U.random_weights(cfg, 8)
    m = _load(tmp_path, cfg, P)
    try:
        for n in (1, 2, 3, 5):
            toks = U.tokens(n, cfg["vocab"], 40 + n)
            s = m.seq_alloc()
            got, _ = m.step_batch([(s, toks, _all(n))])
            assert _err(got, O.forward(cfg, P, toks)) < TOL_F32
            m.seq_free(s)
        # a fresh slot starts from an empty convolution tail although the one before it left its own behind
        toks = U.tokens(4, cfg["vocab"], 50)
        s = m.seq_alloc()
        got = np.concatenate([m.step_batch([(s, [t], [0])])[0] for t in toks])
        assert _err(got, O.forward(cfg, P, toks)) < TOL_F32
    finally:
        m.close()


def test_long_decoding_past_many_windows(tmp_path):
    cfg = U.small_config()                                        # windows of 15 to 70
    P = U.random_weights(cfg, 9)
    toks = U.tokens(230, cfg["vocab"], 9)
    want = O.forward(cfg, P, toks)
    m = _load(tmp_path, cfg, P)
    try:
        s = m.seq_alloc()
        m.step_batch([(s, toks[:10], [])])
        got = np.concatenate([m.step_batch([(s, [toks[p]], [0])])[0] for p in range(10, 230)])
        assert _err(got, want[10:]) < TOL_F32
    finally:
        m.close()


OTHER = {
    "odd width": _one(U.attn(), U.moe(), vocab=53, width=31),
    "everything one": _one(U.attn(heads=1, kv_heads=1, dim=1, vdim=1, conv=1, size=2, rot_dims=0), U.moe(experts=1, top=1, ff=1, shared=1)),
    "one pair per head": _one(U.attn(heads=7, kv_heads=7, dim=2, vdim=1, conv=3, rot_dims=2)),
    "head size 64, value size 128": _one(U.attn(heads=4, kv_heads=2, dim=64, vdim=128, conv=4, rot_dims=32), width=64),
    "head size 128, value size 48": _one(U.attn(heads=2, kv_heads=1, dim=128, vdim=48, conv=4, rot_dims=128), width=64),
    "head size 200, value size 150": _one(U.attn(heads=2, kv_heads=1, dim=200, vdim=150, conv=3, rot_dims=64), width=64),
    "head size 300, value size 260": _one(U.attn(heads=2, kv_heads=1, dim=300, vdim=260, conv=4, rot_dims=300), width=40),
    "twenty query heads on one key head": _one(U.attn(heads=20, kv_heads=1, dim=8, vdim=4, conv=2, rot_dims=4)),
    "no window reached": _one(U.attn(size=5000), U.moe()),
    "seventy experts": _one(U.attn(), U.moe(experts=70, top=6, ff=8, shared=12), width=32),
    "wide rows": _one(U.attn(heads=4, kv_heads=4, dim=40, vdim=60), U.moe(experts=3, top=2, ff=72, shared=200), width=1028, vocab=301),
    "a window longer than the other's, borrowed": U.config([U.layer(U.attn(size=10), U.moe()), U.layer(U.attn(size=120, kv_from=0), U.moe(shared=0))]),
    "saturated norms": _one(U.attn(), U.moe(), embed_scale=60.0),
}


@pytest.mark.parametrize("name", list(OTHER))
def test_other_sizes_whole_portioned_and_decoded(tmp_path, name):
    cfg = OTHER[name]
    P = U.random_weights(cfg, 11)
    toks = U.tokens(150, cfg["vocab"], 11)
    want = O.forward(cfg, P, toks)
    m = _load(tmp_path, cfg, P)
    try:
        a, b = m.seq_alloc(), m.seq_alloc()
        whole, _ = m.step_batch([(a, toks, _all(150))])
        assert _err(whole, want) < TOL_F32
        out, at = [], 0
        for c in [70, 2, 33, 1, 1, 17, 1, 25]:
            out.append(m.step_batch([(b, toks[at:at + c], _all(c))])[0])
            at += c
        assert _err(np.concatenate(out), want) < TOL_F32
    finally:
        m.close()


def test_greedy_generation_through_generate_and_through_the_engine(tmp_path):
    from crane_amd.backend import GenerationConfig
    from crane_amd.engine import GenerationParams, InferenceEngine
    cfg = U.small_config()
    P = U.random_weights(cfg, 12)
    prompts = [U.tokens(n, cfg["vocab"], 60 + i) for i, n in enumerate((9, 70, 3, 25, 40))]
    lens = [12, 6, 20, 9, 15]
    want = [O.greedy(cfg, P, p, n) for p, n in zip(prompts, lens)]
    m = _load(tmp_path, cfg, P, max_seq_len=128, kv_pool_tokens=384, max_seqs=4, prefill_chunk=48)
    try:
        assert m.generate(prompts[0], GenerationConfig.greedy(lens[0]))[len(prompts[0]):] == want[0]
        m.clear_kv_cache()
        eng = InferenceEngine(m, max_running=3)                   # 5 requests, 3 slots, 48-row steps: prompts are fed in portions
        ids = [eng.submit(p, GenerationParams.greedy(n)) for p, n in zip(prompts, lens)]
        toks, done = eng.run_until_idle()
        for rid, w in zip(ids, want):
            assert toks[rid] == w
            assert done[rid].kind == "finished" and done[rid].finish_reason == "length"
        st = eng.stats()
        assert st["completed"] == 5 and st["failed"] == 0 and st["free_pages"] == st["total_pages"]
        # sampled requests run through the same steps and the device sampler
        rid = eng.submit(prompts[3], GenerationParams(max_tokens=8, temperature=0.8, top_p=0.9, top_k=20, seed=5))
        toks, done = eng.run_until_idle()
        assert len(toks[rid]) == 8 and all(0 <= t < cfg["vocab"] for t in toks[rid])
        eng.close()
    finally:
        m.close()


def test_bfloat16_format_against_the_oracle_and_across_schedules(tmp_path):
    cfg = U.small_config()
    P = U.random_weights(cfg, 13)
    toks = U.tokens(100, cfg["vocab"], 13)
    want = O.forward(cfg, P, toks)
    m = _load(tmp_path, cfg, P, dtype="bfloat16")
    try:
        a, b = m.seq_alloc(), m.seq_alloc()
        whole, _ = m.step_batch([(a, toks, _all(100))])
        assert _err_most(whole, want) < TOL_BF16
        out, at = [], 0
        for c in [50, 2, 13, 1, 1, 33]:
            out.append(m.step_batch([(b, toks[at:at + c], _all(c))])[0])
            at += c
        assert _err_most(np.concatenate(out), want) < TOL_BF16
        assert _err_most(np.concatenate(out), whole) < TOL_BF16
    finally:
        m.close()


def test_fork_carries_pages_states_and_convolution_tails(tmp_path):
    cfg = U.small_config()
    P = U.random_weights(cfg, 14)
    toks = U.tokens(80, cfg["vocab"], 14)
    want = O.forward(cfg, P, toks)
    m = _load(tmp_path, cfg, P)
    try:
        a = m.seq_alloc()
        m.step_batch([(a, toks[:37], [])])
        b = m.seq_fork(a)
        ga, _ = m.step_batch([(a, toks[37:], _all(43)), ])
        gb, _ = m.step_batch([(b, toks[37:], _all(43))])
        assert _err(ga, want[37:]) < TOL_F32 and _err(gb, want[37:]) < TOL_F32
        with pytest.raises(Exception):
            m.seq_truncate(a, 10)                                 # a convolution tail cannot be rewound
    finally:
        m.close()


def test_synthetic_registry_model_generates(tmp_path):
    from crane_amd import configs
    from crane_amd.backend import GenerationConfig, Model
    m = Model.synthetic(configs.get_config("tiny-gizezen"), seed=3, max_seq_len=128, max_seqs=2)
    try:
        assert m.num_layers() == 5 and m.vocab_size == 320
        out = m.generate([1, 2, 3, 4, 5], GenerationConfig.greedy(6))
        assert len(out) == 11
        logits = m.forward_step([7, 8, 9], 0)[0, 0]
        assert np.isfinite(logits).all() and int(np.argmax(logits)) == m.forward_step_greedy([7, 8, 9], 0)
        assert m.decode_bytes_per_token(64) > m.weight_bytes() // 8
    finally:
        m.close()


def _wide_config(window=96):
    """Sizes the matrix-core kernels take (head sizes multiples of 16, wide products)."""
    return U.config([U.layer(U.attn(heads=8, kv_heads=2, dim=64, vdim=96, conv=4, size=window, rot_dims=32), U.moe(experts=8, top=2, ff=128, shared=256)),
                     U.layer(U.attn(heads=4, kv_heads=2, dim=64, vdim=96, conv=3, size=window, rot_dims=64, kv_from=0), None),
                     U.layer(U.attn(heads=2, kv_heads=2, dim=112, vdim=64, conv=2, size=window, rot_dims=112, scaling=U.bands()), U.moe(experts=6, top=3, ff=64, shared=128))],
                    vocab=256, width=128)


@pytest.mark.parametrize("dtype,tol,err", [("float32", TOL_F32, _err), ("bfloat16", TOL_BF16, _err_most)])
def test_decode_steps_over_hundreds_of_keys_and_a_long_portion(tmp_path, dtype, tol, err):
    cfg = _wide_config(window=300)
    P = U.random_weights(cfg, 15)
    toks = U.tokens(460, cfg["vocab"], 15)
    want = O.forward(cfg, P, toks)
    m = _load(tmp_path, cfg, P, dtype=dtype)
    try:
        a, b = m.seq_alloc(), m.seq_alloc()
        whole, _ = m.step_batch([(a, toks, _all(460))])               # matrix-core attention (bfloat16)
        assert err(whole, want) < tol
        m.step_batch([(b, toks[:430], [])])
        tail = np.concatenate([m.step_batch([(b, [t], [0])])[0] for t in toks[430:]])     # split keys: a window of 300
        assert err(tail, want[430:]) < tol
    finally:
        m.close()


def test_a_step_larger_than_one_pass_is_cut_into_passes(tmp_path):
    cfg = U.small_config()
    P = U.random_weights(cfg, 16)
    reqs = [U.tokens(n, cfg["vocab"], 70 + i) for i, n in enumerate((75, 3, 41))]
    want = [O.forward(cfg, P, t) for t in reqs]
    m = _load(tmp_path, cfg, P, prefill_chunk=32)
    try:
        seqs = [m.seq_alloc() for _ in reqs]
        out, _ = m.step_batch([(s, t, _all(len(t))) for s, t in zip(seqs, reqs)])
        assert _err(out, np.concatenate(want)) < TOL_F32
    finally:
        m.close()


def test_many_portions_in_one_pass(tmp_path):
    """40 sequences of 20 tokens in one pass, and cut into passes of 128 rows: rows of several sequences side by side in a block."""
    cfg = U.config([U.layer(U.attn(conv=4), None), U.layer(U.attn(conv=6, kv_from=0), U.moe())])
    P = U.random_weights(cfg, 18)
    reqs = [U.tokens(17 + i % 5, cfg["vocab"], 100 + i) for i in range(40)]
    want = np.concatenate([O.forward(cfg, P, t) for t in reqs])
    for chunk in (128, 2048):
        m = _load(tmp_path, cfg, P, max_seqs=40, max_seq_len=64, prefill_chunk=chunk)
        try:
            seqs = [m.seq_alloc() for _ in reqs]
            out, _ = m.step_batch([(s, t, _all(len(t))) for s, t in zip(seqs, reqs)])
            assert _err(out, want) < TOL_F32
            # one more token each: forty single tokens, then their tails serve two more
            nxt = [U.tokens(3, cfg["vocab"], 200 + i) for i in range(40)]
            want2 = [O.forward(cfg, P, t + n)[len(t):] for t, n in zip(reqs, nxt)]
            out, _ = m.step_batch([(s, n[:1], [0]) for s, n in zip(seqs, nxt)])
            assert _err(out, np.stack([w[0] for w in want2])) < TOL_F32
            out, _ = m.step_batch([(s, n[1:], [0, 1]) for s, n in zip(seqs, nxt)])
            assert _err(out, np.concatenate([w[1:] for w in want2])) < TOL_F32
        finally:
            m.close()


def test_matrix_core_attention_of_prompt_passes_against_the_plain_kernel(tmp_path):
    cfg = _wide_config()
    P = U.random_weights(cfg, 17)
    toks = U.tokens(300, cfg["vocab"], 17)
    want = O.forward(cfg, P, toks)
    m = _load(tmp_path, cfg, P, dtype="bfloat16")
    try:
        a, b = m.seq_alloc(), m.seq_alloc()
        fast, _ = m.step_batch([(a, toks[:130], _all(130))])
        fast2, _ = m.step_batch([(a, toks[130:], _all(170))])        # a portion whose keys lie in earlier pages
        fast = np.concatenate([fast, fast2])
        m.debug_set("lay_attn_mfma", 0)
        plain, _ = m.step_batch([(b, toks, _all(300))])
        assert _err_most(fast, want) < TOL_BF16 and _err_most(plain, want) < TOL_BF16
        assert _err_most(fast, plain) < 3e-2
    finally:
        m.close()


def _drawn_config(seed):
    """A model of this design with layer order, loans, sizes, windows and constants drawn from the seed."""
    rs = np.random.RandomState(400 + seed)
    pick = lambda *xs: xs[rs.randint(len(xs))]
    layers = []

    def mlp():
        if rs.rand() < 0.2:
            return None
        experts = pick(3, 4, 8, 12)
        return U.moe(experts=experts, top=rs.randint(1, min(experts, 4) + 1), ff=pick(32, 72, 96), shared=pick(0, 40, 128))

    for i in range(rs.randint(3, 7)):
        own = [j for j, ly in enumerate(layers) if "kv_from" not in ly["mixer"]]
        scaling = pick(None, U.bands(pick(2.0, 8.0), pick(0.5, 1.0), pick(3.0, 4.0), pick(64, 256, 1000)))
        common = dict(conv=pick(1, 2, 3, 4, 5), size=pick(17, 40, 64, 80, 136), base=pick(500.0, 1e4, 1e6), scaling=scaling, scale=pick(None, 0.1, 0.5))
        if own and rs.rand() < 0.45:
            j = own[rs.randint(len(own))]
            src = layers[j]["mixer"]
            mx = U.attn(heads=src["kv_heads"] * pick(1, 2, 3), kv_heads=src["kv_heads"], dim=src["dim"], vdim=src["vdim"],
                        rot_dims=src["rot"]["dims"], kv_from=j, **common)
        else:
            g, dim = pick(1, 2, 3), pick(16, 24, 32, 48, 64, 96)
            mx = U.attn(heads=g * pick(1, 2, 4), kv_heads=g, dim=dim, vdim=pick(16, 32, 40, 80), rot_dims=pick(dim, dim // 2, 0), **common)
        layers.append(U.layer(mx, mlp()))
    return U.config(layers, vocab=pick(97, 256, 601), width=pick(96, 120, 192, 240), eps=pick(1e-6, 1e-5, 1e-4), mult=pick(0.2, 0.5, 1.0), embed_scale=pick(1.0, 4.0, 12.0))


@pytest.mark.parametrize("seed", range(8))
def test_drawn_models_whole_in_portions_and_decoded_in_both_formats(tmp_path, seed):
    cfg = _drawn_config(seed)
    P = U.random_weights(cfg, 30 + seed)
    toks = U.tokens(170, cfg["vocab"], 30 + seed)
    want = O.forward(cfg, P, toks)
    for dtype, tol, err in (("float32", TOL_F32, _err), ("bfloat16", TOL_BF16, _err_most)):
        m = _load(tmp_path, cfg, P, dtype=dtype)
        try:
            a, b = m.seq_alloc(), m.seq_alloc()
            whole, _ = m.step_batch([(a, toks, _all(170))])
            assert err(whole, want) < tol, (dtype, "whole")
            out, at = [], 0
            for c in [70, 2, 33, 1, 1, 17, 1, 25, 1, 1, 18]:
                out.append(m.step_batch([(b, toks[at:at + c], _all(c))])[0])
                at += c
            assert at == 170 and err(np.concatenate(out), want) < tol, (dtype, "portions")
        finally:
            m.close()


def test_a_trace_of_mixed_steps_replayed_by_the_command_line_runner(tmp_path):
    """bin/trace_run on a small model: five requests over four slots and a pool of 7 pages (their sum: 9), portions beside single tokens,
    requests that end and whose pages and slots the next ones take."""
    import json
    import os
    import subprocess
    import sys
    cfg = U.small_config()
    P = U.random_weights(cfg, 19)
    ckpt = U.write_checkpoint(str(tmp_path / "ckpt"), cfg, P)
    reqs = {n: U.tokens(k, cfg["vocab"], 80 + i) for i, (n, k) in enumerate((("a", 90), ("b", 7), ("c", 130), ("d", 40), ("e", 66)))}
    want = {n: O.forward(cfg, P, t) for n, t in reqs.items()}
    plan = [[("a", 50), ("b", 2)], [("a", 1), ("b", 1), ("c", 64)], [("c", 2), ("a", 39), ("b", 4), ("d", 30)], [("d", 10), ("c", 60)],
            [("e", 3)], [("e", 62), ("c", 0)], [("e", 1)]]
    at = {n: 0 for n in reqs}
    lines, asked = [], []
    for n_step, step in enumerate(plan):
        entries, end, rows = [], [], []
        for n, c in step:
            c = c or len(reqs[n]) - at[n]
            wanted = sorted({0, c - 1, c // 2})
            entries.append(dict(id=n, tokens=reqs[n][at[n]:at[n] + c], want=wanted))
            rows += [(n, at[n] + k) for k in wanted]
            at[n] += c
            if at[n] == len(reqs[n]):
                end.append(n)
        lines.append(json.dumps(dict(step=n_step, entries=entries, end=end)))
        asked.append(rows)
    assert all(at[n] == len(reqs[n]) for n in reqs)
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    for dtype, tol, err in (("float32", TOL_F32, _err), ("bfloat16", 4 * TOL_BF16, _err_most)):       # (few rows, drawn from five requests)
        out = tmp_path / ("out_" + dtype)
        run = subprocess.run([sys.executable, os.path.join(root, "bin", "trace_run"), "--model", ckpt, "--dtype", dtype, "--out", str(out), "--max-tokens", "448"],
                             input="\n".join(lines) + "\n", capture_output=True, text=True, timeout=600)
        assert run.returncode == 0, run.stderr[-2000:]
        assert [x for x in run.stdout.split("\n") if x.startswith("done")] == ["done %d" % i for i in range(len(plan))]
        got = np.concatenate([np.fromfile(out / ("%d.f32" % i), "<f4").reshape(-1, cfg["vocab"]) for i in range(len(plan))])
        ref = np.stack([want[n][p] for rows in asked for n, p in rows])
        assert got.shape == ref.shape and err(got, ref) < tol, dtype
