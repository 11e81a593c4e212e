"""Bubetar models on the device against the float64 oracle (oracle/layered.py): attention beside a recurrence in one layer
(gates, sinks, windows, keys as values, rotations of either layout; lightning attention, the delta rule with a decay per
channel), latent attention over everything before, norms on both sides of a sublayer; prompts, decoding, portions, mixed
batches, reuse of pages and state slots, far keys and old states, and generation through the framework's own entry points."""
import copy

import numpy as np
import pytest

import layered_common as lc
from gpu_common import ops
from layered_common import oracle
from test_gpu_layered import F32_TOL, oracle_greedy, step_logits, tables_of, whole

pytestmark = pytest.mark.gpu

BF16_TOL = 0.1


@pytest.fixture
def tune():
    from fandhe_ai_amd.capi import lib
    used = []

    def set_key(key, value):
        used.append(key)
        assert lib.fa_set_tuning(key, value) == 0
    yield set_key
    for key in used:
        lib.fa_set_tuning(key, 0)


def tolerance(dtype):
    return F32_TOL if dtype == "float32" else BF16_TOL


def left(**kw):
    return lc.parallel(left=lc.gated_left(**kw))


def right(**kw):
    return lc.parallel(right=lc.lightning_right(**kw))


def left_2(**kw):
    return lc.parallel_2(left=lc.key_value_left(**kw))


def right_2(**kw):
    return lc.parallel_2(right=lc.channel_right(**kw))


MECHANISMS = {
    "gated attention and lightning": [lc.parallel()],
    "gated, a key head per query head, all rotated": [left(heads=3, kv_heads=3, dim=16, vdim=16, rot=16)],
    "gated, one key head, one rotated pair, sizes of no multiple": [left(heads=5, kv_heads=1, dim=9, vdim=7, rot=2)],
    "gated, an odd number of rotated pairs": [left(dim=24, rot=6, vdim=20)],
    "gated 64 128": [left(heads=4, kv_heads=2, dim=48, vdim=128, rot=20)],
    "gated 128 64": [left(heads=8, kv_heads=4, dim=128, vdim=40, rot=64)],
    "gated 128 128": [left(heads=4, kv_heads=1, dim=128, vdim=128, rot=128)],
    "gated 256": [left(heads=2, kv_heads=1, dim=130, vdim=200, rot=34)],
    "gated beyond the matrix-core sizes": [left(heads=2, kv_heads=1, dim=300, vdim=260, rot=100)],
    "gated, twenty query heads a key head": [left(heads=40, kv_heads=2, dim=8, vdim=12, rot=4)],
    "lightning, one head of one dim": [right(heads=1, dim=1, vdim=1)],
    "lightning, odd sizes": [right(heads=5, dim=9, vdim=7)],
    "lightning 128": [right(heads=4, dim=128, vdim=128)],
    "lightning 256": [right(heads=2, dim=256, vdim=48)],
    "lightning wide": [right(heads=2, dim=130, vdim=260)],
    "lightning, decays from nothing to all": [right(heads=4, dim=16, vdim=16, decay=[0.0, 1.0, 0.02, 0.9995])],
    "key values and channel decays": [lc.parallel_2()],
    "key values, all rotated, no scaling": [left_2(dim=16, rot=16, scaling=None)],
    "key values, one rotated pair, sizes of no multiple": [left_2(heads=5, kv_heads=1, dim=9, rot=2, window=5)],
    "key values, a long stretch": [left_2(dim=32, rot=32, base=80.0, scaling=(20.0, 0.5, 9.0, 40))],
    "key values 64": [left_2(heads=4, kv_heads=4, dim=64, rot=24, window=37)],
    "key values 128": [left_2(heads=6, kv_heads=2, dim=128, rot=64, window=21)],
    "key values 256": [left_2(heads=2, kv_heads=1, dim=200, rot=88, window=16)],
    "key values beyond the matrix-core sizes": [left_2(heads=2, kv_heads=2, dim=270, rot=8, window=9)],
    "window of one": [left_2(window=1)],
    "window longer than the sequence": [left_2(window=4096)],
    "channel decays, a key head per head": [right_2(heads=3, kv_heads=3, dim=16, vdim=32, conv=3)],
    "channel decays, one key head, no convolution history": [right_2(heads=5, kv_heads=1, dim=9, vdim=7, conv=1)],
    "channel decays 128": [right_2(heads=4, kv_heads=2, dim=128, vdim=128, conv=4)],
    "channel decays 256": [right_2(heads=2, kv_heads=1, dim=256, vdim=48, conv=5)],
    "channel decays wide": [right_2(heads=2, kv_heads=1, dim=130, vdim=260, conv=2)],
    "latent": [lc.open_latent()],
    "latent one head, tiny sizes": [lc.open_latent(heads=1, dim=1, rot=2, vdim=1, q_rank=3, kv_rank=5)],
    "latent 512": [lc.open_latent(heads=20, dim=128, rot=64, vdim=128, q_rank=192, kv_rank=512)],
    "latent middle sizes": [lc.open_latent(heads=5, dim=70, rot=40, vdim=100, q_rank=64, kv_rank=200)],
    "feed-forward": [lc.open_latent(mlp=lc.dense(77))],
    "all": [lc.parallel(mlp=lc.dense()), lc.parallel_2(mlp=lc.dense(33)), lc.open_latent(mlp=lc.dense(64)), lc.parallel_2(), lc.open_latent(kv_rank=60), lc.parallel()],
}


def portions_of(dec, toks, sizes, slots=None):
    """All positions' logits of a sequence fed in portions of the given sizes, over and over."""
    dec.set_sequences(tables_of(dec, 1), [0])
    got, at, i = [], 0, 0
    while at < len(toks):
        n = min(sizes[i % len(sizes)], len(toks) - at)
        got.append(dec.forward([toks[at:at + n]], [list(range(n))]))
        at, i = at + n, i + 1
    return np.concatenate(got)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", sorted(MECHANISMS))
def test_mechanism_prompt_then_decode(name, dtype):
    """A prompt in one pass, every position's logits; then the same tokens with the last ones decoded one by one."""
    cfg = lc.bubetar(MECHANISMS[name])
    w = lc.weights(cfg, 11)
    toks = lc.tokens(cfg, 75, 3)
    want = oracle.forward(cfg, w, toks)
    dec = lc.make_decoder(ops(), cfg, w, dtype)
    assert lc.error(whole(dec, toks), want) < tolerance(dtype)
    assert lc.error(portions_of(dec, toks, (37,) + (1,) * 38), want) < tolerance(dtype)
    dec.close()


FORMS = {"attention plain": (33, 1), "attention few rows": (33, 2), "attention many rows": (33, 3), "attention, keys split further": (34, 8),
         "latent plain": (30, 1), "latent absorbed": (30, 2), "latent expanded": (30, 3), "recurrence token by token": (31, 1), "small tiles": (29, 2)}
FORM_LAYERS = {
    "all": MECHANISMS["all"],
    "large sizes": [lc.parallel(lc.gated_left(12, 3, 128, 128, 64), lc.lightning_right(3, 128, 128), mlp=lc.dense(272)),
                    lc.parallel_2(lc.key_value_left(12, 3, 128, 64, 150), lc.channel_right(4, 2, 128, 128)), lc.open_latent(20, 128, 64, 128, 64, 512)],
}


@pytest.mark.parametrize("form", sorted(FORMS))
@pytest.mark.parametrize("name", sorted(FORM_LAYERS))
def test_every_kernel_form_gives_the_oracles_logits(name, form, tune):
    """bf16: prompts longer than a tile, portions behind cached tokens, and decoding, on every form of the kernels."""
    tune(*FORMS[form])
    cfg = lc.bubetar(FORM_LAYERS[name], width=128, ranks=(16, 24))
    w = lc.weights(cfg, 23)
    toks = lc.tokens(cfg, 420, 3)
    want = oracle.forward(cfg, w, toks)
    dec = lc.make_decoder(ops(), cfg, w, "bfloat16")
    assert lc.error(whole(dec, toks), want) < BF16_TOL
    got = portions_of(dec, toks[:400], (45, 310, 17) + (1,) * 28)
    assert lc.error(got, want[:400]) < BF16_TOL
    dec.close()


def test_residual_stream_after_every_layer():
    cfg = lc.bubetar(MECHANISMS["all"])
    w = lc.weights(cfg, 2)
    toks = lc.tokens(cfg, 30, 2)
    want = []
    oracle.forward(cfg, w, toks, want)
    dec = lc.make_decoder(ops(), cfg, w)
    dec.set_sequences(tables_of(dec, 1), [0])
    _, got = dec.forward([toks], [[]], residuals=True)
    for i, (g, r) in enumerate(zip(got, want)):
        assert np.abs(g - r).max() < 2e-4 * np.abs(r).max(), i
    dec.close()


@pytest.mark.parametrize("width,vocab,block_size,ranks", [(64, 96, 16, (1, 1)), (129, 50, 64, (3, 40)), (320, 1000, 1, (70, 2)), (1500, 40, 256, (16, 8))])
def test_other_widths_vocabularies_pages_and_ranks(width, vocab, block_size, ranks):
    cfg = lc.bubetar(MECHANISMS["all"][:3], width=width, vocab=vocab, eps=3e-4, softcap=3.0, scale=1.9, ranks=ranks)
    w = lc.weights(cfg, 4)
    toks = lc.tokens(cfg, 60, 4)
    want = oracle.forward(cfg, w, toks)
    for dtype, as_bf16 in (("float32", True), ("float32", False), ("bfloat16", True)):
        dec = lc.make_decoder(ops(), cfg, w, dtype, as_bf16=as_bf16, block_size=block_size)
        assert lc.error(whole(dec, toks), want) < tolerance(dtype)
        dec.close()


@pytest.mark.parametrize("use_graph", [False, True])
def test_steps_continue_a_prompt_pass(use_graph):
    cfg = lc.bubetar(MECHANISMS["all"])
    w = lc.weights(cfg, 7)
    toks = lc.tokens(cfg, 90, 7)
    want = oracle.forward(cfg, w, toks)
    dec = lc.make_decoder(ops(), cfg, w)
    for start in (1, 34):
        dec.set_sequences(tables_of(dec, 1), [0])
        dec.prefill([toks[:start]])
        assert lc.error(dec.logits(), want[start - 1:start]) < F32_TOL
        assert dec.tokens()[0] == dec.logits()[0].argmax()
        assert lc.error(step_logits(dec, toks, start, use_graph), want[start:]) < F32_TOL
        assert dec.seq_lens()[0] == len(toks)
    dec.close()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_portions_of_any_size_leave_the_same_logits(dtype):
    cfg = lc.bubetar(MECHANISMS["all"])
    w = lc.weights(cfg, 8)
    toks = lc.tokens(cfg, 230, 8)
    want = oracle.forward(cfg, w, toks)
    dec = lc.make_decoder(ops(), cfg, w, dtype)
    assert lc.error(whole(dec, toks), want) < tolerance(dtype)
    for sizes in ((2,), (3, 2), (11, 12, 13), (16,), (17, 15), (32,), (33, 31), (64,), (65, 63, 2), (7, 128), (100, 1, 1, 2)):
        assert lc.error(portions_of(dec, toks, sizes), want) < tolerance(dtype), sizes
    dec.close()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_mixed_batches_match_each_request_alone(dtype):
    """Portions of some beside single tokens of others, rows changing places, requests left out of steps."""
    cfg = lc.bubetar(MECHANISMS["all"])
    w = lc.weights(cfg, 9)
    reqs = {r: lc.tokens(cfg, n, 20 + i) for i, (r, n) in enumerate((("a", 260), ("b", 33), ("c", 90), ("d", 5)))}
    dec = lc.make_decoder(ops(), cfg, w, dtype)
    rng = np.random.default_rng(3)
    from fandhe_ai_amd.scheduler import PortionBatcher
    b = PortionBatcher(dec)
    at = dict.fromkeys(reqs, 0)
    got = {r: [] for r in reqs}
    while any(at[r] < len(t) for r, t in reqs.items()):
        names = [r for r in reqs if at[r] < len(reqs[r]) and rng.random() < 0.8]
        rng.shuffle(names)
        entries = []
        for r in names:
            n = min(int(rng.choice([1, 1, 2, 3, 16, 70])), len(reqs[r]) - at[r])
            entries.append((r, reqs[r][at[r]:at[r] + n], list(range(n))))
        if not entries:
            continue
        rows = b.feed(entries)
        for r, t, _ in entries:
            got[r].append(rows[:len(t)])
            rows = rows[len(t):]
            at[r] += len(t)
    for r, t in reqs.items():
        assert lc.error(np.concatenate(got[r]), oracle.forward(cfg, w, t)) < tolerance(dtype), r
    dec.close()


def test_freed_pages_and_slots_carry_nothing_over():
    """A pool of five pages and two states: every later request runs on what earlier ones left behind, in another order."""
    cfg = lc.bubetar(MECHANISMS["all"])
    w = lc.weights(cfg, 10)
    dec = lc.make_decoder(ops(), cfg, w, max_tokens=80, max_batch=2, state_slots=2)
    from fandhe_ai_amd.scheduler import PortionBatcher
    b = PortionBatcher(dec)
    for i, n in enumerate((70, 3, 40, 80, 1, 33)):
        toks = lc.tokens(cfg, n, 50 + i)
        first = (n // 2 + 1, 1, 2)[i % 3]
        got = b.feed([(i, toks[:first], list(range(first)))])
        for t in toks[first:n // 2]:
            got = np.concatenate([got, b.feed([(i, [t], [0])])])
        rest = toks[max(first, n // 2):]
        if rest:
            got = np.concatenate([got, b.feed([(i, rest, list(range(len(rest))))])])
        assert lc.error(got, oracle.forward(cfg, w, toks)) < F32_TOL, i
        b.release(i)
        if i % 2:
            b.feed([("takes a page %d" % i, [1], [])])
            b.release("takes a page %d" % i)
    assert b.free_pages() == 5
    dec.close()


SPECIAL = 39


def standing_out(layer, at, n, latent=False):
    """A model of one layer whose queries are all alike and in which one token's key wins every score that sees it by far; the
    sequence holds it at the places `at`.  Channel 0 of the embedding is steady, channel 1 tells that token from the others."""
    cfg = lc.bubetar([layer], width=96, vocab=40, eps=1e-6)
    w = lc.weights(cfg, 12)
    rng = np.random.default_rng(1)
    w["embed"][:, 0], w["embed"][:, 1] = 5.0, 5.0
    w["embed"][SPECIAL, 1] = -5.0
    w["l0.norm1"][:] = 1.0
    mx = layer["mixer"]
    if latent:
        p, H, d, r = "l0.mix.", mx["heads"], mx["dim"], mx["kv_rank"]
        w[p + "dq"] = lc.bf16_round((0.01 * rng.normal(size=w[p + "dq"].shape)).astype(np.float32))
        w[p + "dq"][:, 0] = 1.0                               # the query latent: all ones
        w[p + "dq.norm"][:] = 1.0
        w[p + "dkv"] = lc.bf16_round((0.05 * rng.normal(size=w[p + "dkv"].shape)).astype(np.float32))
        w[p + "dkv"][:r, 1] = -1.0                            # the key latent: plus or minus ones
        uk, uq = rng.normal(size=(H, d, r)), rng.normal(size=(H, d + mx["rot_dim"], mx["q_rank"])) * 0.01
        uq[:, :d] += (uk.sum(axis=2) / np.abs(uk.sum(axis=2)).sum(axis=1, keepdims=True) / d ** 0.5)[:, :, None]
        w[p + "uk"], w[p + "uq"] = (lc.bf16_round(a.reshape(-1, a.shape[2]).astype(np.float32)) for a in (uk, uq))
    else:
        p, a = "l0.mix.left.", mx["left"]
        way = np.where(rng.random(a["dim"]) < 0.5, -1.0, 1.0)
        way[[0, 1] if layer["type"] == "parallel" else [0, a["rot"]["dims"] // 2]] = 0.0           # turned with the position
        q, k = 0.02 * rng.normal(size=w[p + "q"].shape), 0.02 * rng.normal(size=w[p + "k"].shape)
        q[:, 0], k[:, 1] = np.tile(way, a["heads"]), -np.tile(way, a["kv_heads"])
        w[p + "q"], w[p + "k"] = lc.bf16_round(q.astype(np.float32)), lc.bf16_round(k.astype(np.float32))
        for name in ("q.norm", "k.norm"):
            if p + name in w:
                w[p + name][:] = 1.0
    toks = [int(t) for t in rng.integers(0, SPECIAL, n)]
    for i in at:
        toks[i] = SPECIAL
    return cfg, w, toks


def check_standing_out(cfg, w, toks, dtype, cuts):
    want = oracle.forward(cfg, w, toks)
    dec = lc.make_decoder(ops(), cfg, w, dtype, max_tokens=768)
    assert lc.error(whole(dec, toks), want) < tolerance(dtype)
    for cut in cuts:
        mid = max(cut, len(toks) - 60)
        got = portions_of(dec, toks, (cut, mid - cut) + (1,) * 60 if mid > cut else (cut,) + (1,) * 60)
        assert lc.error(got, want) < tolerance(dtype), cut
    dec.close()


FAR = {
    "gated 64, the first token": (lc.parallel(lc.gated_left(4, 2, 16, 16, 2, 2.0), scales=(1.0, 0.2)), (0,), 400, False),
    "gated 64, page and tile borders": (lc.parallel(lc.gated_left(4, 1, 16, 8, 2, 2.0), scales=(1.0, 0.2)), (63, 300), 420, False),
    "gated 128": (lc.parallel(lc.gated_left(2, 1, 128, 128, 2, 0.4), scales=(1.0, 0.2)), (31, 511), 640, False),
    "gated 256": (lc.parallel(lc.gated_left(4, 4, 200, 96, 2, 0.4), scales=(1.0, 0.2)), (32, 33), 150, False),
    "latent 64": (lc.open_latent(4, 16, 4, 16, 24, 44, 2.0), (0, 17), 400, True),
    "latent 512": (lc.open_latent(3, 16, 4, 16, 24, 512, 1.0), (63,), 500, True),
}


@pytest.mark.parametrize("name", sorted(FAR))
@pytest.mark.parametrize("dtype,form", [("float32", 0), ("bfloat16", 0), ("bfloat16", 1), ("bfloat16", 2), ("bfloat16", 3)])
def test_a_far_key_that_stands_out(name, dtype, form, tune):
    """Seen from its own position to the end, hundreds of tokens on, in prompts, portions and decoding."""
    layer, at, n, latent = FAR[name]
    tune(30 if latent else 33, form)
    cfg, w, toks = standing_out(layer, at, n, latent)
    want, hidden = oracle.forward(cfg, w, toks), oracle.forward(cfg, w, [5 if t == SPECIAL else t for t in toks])
    for p in (at[0], n - 1):                                  # far beyond the tolerance: at its own place and at the far end
        assert lc.error(hidden[p:p + 1], want[p:p + 1]) > 0.2, p
    check_standing_out(cfg, w, toks, dtype, (1, at[-1] + 1, n - 40))


@pytest.mark.parametrize("dtype,form", [("float32", 0), ("bfloat16", 0), ("bfloat16", 1), ("bfloat16", 2), ("bfloat16", 3)])
@pytest.mark.parametrize("dim,share,window", [(16, 2, 1), (16, 1, 16), (40, 3, 17), (128, 1, 33), (128, 4, 150), (200, 2, 64)])
def test_window_edges(dim, share, window, dtype, form, tune):
    """The key that wins shows exactly as long as the window holds it; what is left without it goes to the sink."""
    tune(33, form)
    layer = lc.parallel_2(lc.key_value_left(2 * share, 2, dim, 2, window, 32.0 / dim), scales=(1.0, 0.2))
    n = 3 * window + 40
    at = (0, 15, 16, window + 20)
    cfg, w, toks = standing_out(layer, at, n)
    want = oracle.forward(cfg, w, toks)
    for off in (-1, 1):                                       # a window one off would be seen, far beyond the tolerance
        if window + off < 1:
            continue
        wrong = copy.deepcopy(cfg)
        wrong["layers"][0]["mixer"]["left"]["mask"]["size"] = window + off
        assert lc.error(oracle.forward(wrong, w, toks), want) > 0.3
    check_standing_out(cfg, w, toks, dtype, (1, window, window + 21))


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_sinks_from_nothing_to_everything(dtype):
    """One head's sink is far below its scores, one about them, one far above; the windows hold few keys and many."""
    for window in (3, 500):
        cfg = lc.bubetar([lc.parallel_2(lc.key_value_left(6, 3, 20, 8, window))])
        w = lc.weights(cfg, 31)
        w["l0.mix.left.sink"][:] = [-100.0, -3.0, 0.0, 2.5, 9.0, 200.0]
        toks = lc.tokens(cfg, 330, 31)
        want = oracle.forward(cfg, w, toks)
        gone = dict(w, **{"l0.mix.left.sink": np.full(6, -1e9, np.float32)})
        assert lc.error(oracle.forward(cfg, gone, toks), want) > 3 * BF16_TOL
        dec = lc.make_decoder(ops(), cfg, w, dtype)
        assert lc.error(whole(dec, toks), want) < tolerance(dtype)
        assert lc.error(portions_of(dec, toks, (200, 90) + (1,) * 40), want) < tolerance(dtype)
        dec.close()


@pytest.mark.parametrize("kind", ["lightning", "channel"])
def test_what_was_written_long_ago_is_read_back_from_the_state(kind):
    """Decays near one and one token among the others that writes much (a large key; a full write where the others hardly write):
    what it left is read hundreds of tokens on, through portions and through decoding."""
    if kind == "lightning":
        layer = lc.parallel(lc.gated_left(2, 1, 8, 8, 2), lc.lightning_right(2, 32, 16, [1.0, 0.9999]), (0.0, 1.0))
    else:
        layer = lc.parallel_2(lc.key_value_left(2, 1, 8, 2, 3), lc.channel_right(2, 1, 32, 16, 2), (0.0, 1.0))
    cfg = lc.bubetar([layer], width=64, vocab=40)
    w = lc.weights(cfg, 13)
    w["embed"][:, 1] = 5.0
    w["embed"][SPECIAL, 1] = -5.0
    w["l0.norm1"][1] = 1.0
    if kind == "channel":
        w["l0.mix.right.A_log"][:] = -12.0
        w["l0.mix.right.b"][:, 1] = -3.0
    else:
        w["l0.mix.right.k"][:, 1] = -3.0
    n = 400
    toks = [t % SPECIAL for t in lc.tokens(cfg, n, 1)]
    toks[3] = SPECIAL
    want = oracle.forward(cfg, w, toks)
    other = list(toks)
    other[3] = 17
    for p in (5, n - 1):
        assert lc.error(oracle.forward(cfg, w, other)[p:p + 1], want[p:p + 1]) > 1000 * F32_TOL
    dec = lc.make_decoder(ops(), cfg, w)
    assert lc.error(whole(dec, toks), want) < F32_TOL
    assert lc.error(portions_of(dec, toks, (150, 35, 35, 35, 35, 35, 35) + (1,) * 40), want) < F32_TOL
    dec.close()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_strong_and_uneven_decays(dtype):
    """Channels that forget within a token beside channels that keep everything, heads alike: products of decays that no
    quotient of running products could hold."""
    cfg = lc.bubetar([lc.parallel_2(right=lc.channel_right(4, 2, 24, 20, 3), scales=(0.3, 1.5)), lc.parallel_2(right=lc.channel_right(2, 2, 64, 64))])
    w = lc.weights(cfg, 14)
    rng = np.random.default_rng(14)
    for i, heads in ((0, 4), (1, 2)):
        p = "l%d.mix.right." % i
        w[p + "A_log"][:] = lc.bf16_round(np.log([300.0, 20.0, 3.0, 0.001][:heads]).astype(np.float32))
        w[p + "dt_bias"][:] = lc.bf16_round(rng.uniform(-12.0, 6.0, w[p + "dt_bias"].shape).astype(np.float32))
        w[p + "a2"][:] *= 2.0
    toks = lc.tokens(cfg, 150, 14)
    want = oracle.forward(cfg, w, toks)
    dec = lc.make_decoder(ops(), cfg, w, dtype)
    for sizes in ((150,), (33, 17), (12, 11), (1,)):
        assert lc.error(portions_of(dec, toks, sizes), want) < tolerance(dtype), sizes
    dec.close()


def test_first_tokens():
    cfg = lc.bubetar(MECHANISMS["all"])
    w = lc.weights(cfg, 14)
    dec = lc.make_decoder(ops(), cfg, w)
    for n in range(1, 6):
        toks = lc.tokens(cfg, n, n)
        want = oracle.forward(cfg, w, toks)
        assert lc.error(whole(dec, toks), want) < F32_TOL
        assert lc.error(portions_of(dec, toks, (1,)), want) < F32_TOL
    dec.close()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_long_decoding_of_unequal_requests(dtype):
    """Three rows decoded together from graphs for 150 steps, windows and pages passing over decoded tokens."""
    cfg = lc.bubetar(MECHANISMS["all"])
    w = lc.weights(cfg, 15)
    rows = [lc.tokens(cfg, n + 150, 60 + n) for n in (1, 18, 300)]
    dec = lc.make_decoder(ops(), cfg, w, dtype, max_tokens=1500)
    dec.set_sequences(tables_of(dec, 3), [0, 0, 0])
    dec.prefill_padded([r[:-150] for r in rows])
    got = [[] for _ in rows]
    for t in range(150):
        dec.set_tokens([r[len(r) - 150 + t] for r in rows])
        dec.step()
        for g, x in zip(got, dec.logits()):
            g.append(x)
    for g, r in zip(got, rows):
        assert lc.error(g, oracle.forward(cfg, w, r)[-150:]) < tolerance(dtype)
    dec.close()


def test_many_rows_decode_together():
    """A step of a hundred rows at two kinds of positions."""
    cfg = lc.bubetar(MECHANISMS["all"])
    w = lc.weights(cfg, 16)
    toks = lc.tokens(cfg, 22, 5)
    want = oracle.forward(cfg, w, toks)
    for dtype in ("float32", "bfloat16"):
        dec = lc.make_decoder(ops(), cfg, w, dtype, max_tokens=3200, max_batch=100)
        dec.set_sequences(tables_of(dec, 100), [0] * 100)
        dec.forward([toks[:20] if b % 3 else toks[:1] for b in range(100)])
        got = dec.forward([[toks[20]] if b % 3 else [toks[1]] for b in range(100)], [[0]] * 100)
        assert lc.error(got, np.array([want[20] if b % 3 else want[1] for b in range(100)])) < tolerance(dtype)
        dec.close()


def test_greedy_generation_and_scheduler():
    """generate() and the batch scheduler against greedy decoding with the oracle; more requests than rows, pages or states."""
    from fandhe_ai_amd.scheduler import BatchScheduler, GenerateConfig, InvalidArgument, SamplingStrategy, SchedulerLimits, generate, generate_speculative
    cfg = lc.bubetar(MECHANISMS["all"][:3])
    w = lc.weights(cfg, 16)
    prompts = [lc.tokens(cfg, n, 70 + n) for n in (3, 20, 9, 31, 1)]
    want = [oracle_greedy(cfg, w, p, len(p) + 12) for p in prompts]
    dec = lc.make_decoder(ops(), cfg, w, max_tokens=112, max_batch=3, state_slots=3)
    for p, t in zip(prompts, want):
        assert generate(dec, np.array(p), GenerateConfig(len(t), SamplingStrategy.Greedy())).tolist() == t
    sched = BatchScheduler(dec, SchedulerLimits(3, 8, 64))
    ids = [sched.submit(np.array(p), GenerateConfig(len(t), SamplingStrategy.Greedy())) for p, t in zip(prompts, want)]
    done = {}
    for _ in range(200):
        sched.step()
        done.update(sched.take_finished())
        assert sched.take_failed() == []
        if len(done) == len(ids):
            break
    assert [done[i].tolist() for i in ids] == want
    with pytest.raises(InvalidArgument, match="recurrent"):
        generate_speculative(dec, dec, np.array(prompts[1]), GenerateConfig(len(want[1]), SamplingStrategy.Greedy()), 3)
    dec.close()


def test_long_prompts_run_in_several_internal_passes(tune):
    cfg = lc.bubetar(MECHANISMS["all"])
    w = lc.weights(cfg, 18)
    rows = [lc.tokens(cfg, n, 80 + n) for n in (150, 40, 90)]
    want = [oracle.forward(cfg, w, r) for r in rows]
    dec = lc.make_decoder(ops(), cfg, w)
    tune(28, 64)
    dec.set_sequences(tables_of(dec, 3), [0, 0, 0])
    got = dec.forward(rows, [[0, 63, 64, 149], [39], [1, 88]])
    ref = np.concatenate([want[0][[0, 63, 64, 149]], want[1][[39]], want[2][[1, 88]]])
    assert lc.error(got, ref) < F32_TOL
    dec.set_sequences(tables_of(dec, 3), [0, 0, 0])
    dec.prefill_padded(rows)
    assert lc.error(dec.logits(), np.array([x[-1] for x in want])) < F32_TOL
    dec.close()


def test_checkpoint_folder_trace_and_command_line(tmp_path, capsys):
    """A folder like any other: the ranks of the low-rank projections come from the weights, and norms of a feed-forward that a
    layer has not are passed over."""
    import io
    import json
    import types
    import fandhe_ai_amd as fa
    from fandhe_ai_amd import __main__ as cli
    from fandhe_ai_amd import trace
    cfg = lc.bubetar(MECHANISMS["all"], ranks=(5, 9))
    w = lc.weights(cfg, 21)
    (tmp_path / "config.json").write_text(json.dumps({k: v for k, v in cfg.items() if not k.startswith("_")}))
    typed = {n: fa.safetensors_io.TypedTensor("BF16", a.shape, (a.view(np.uint32) >> 16).astype(np.uint16)) for n, a in w.items()}
    typed["l3.norm2"] = typed["l3.norm2b"] = typed["l3.norm1"]
    fa.safetensors_io.save_safetensors_typed(str(tmp_path / "model.safetensors"), typed)
    toks = lc.tokens(cfg, 40, 9)
    want = oracle.forward(cfg, w, toks)
    steps = [{"step": 0, "entries": [{"id": "x", "tokens": toks[:30], "want": [0, 29]}], "end": []},
             {"step": 1, "entries": [{"id": "y", "tokens": toks[:5], "want": []}, {"id": "x", "tokens": toks[30:], "want": [9]}], "end": ["x"]}]
    args = types.SimpleNamespace(model=str(tmp_path), dtype="float32", out=str(tmp_path), max_tokens=128, device=0)
    assert trace.run(args, io.StringIO("\n".join(json.dumps(s) for s in steps))) == 0
    assert capsys.readouterr().out.split("\n")[:2] == ["done 0", "done 1"]
    got = np.concatenate([np.fromfile(tmp_path / ("%d.f32" % i), "<f4").reshape(-1, cfg["vocab"]) for i in (0, 1)])
    assert lc.error(got, want[[0, 29, 39]]) < F32_TOL
    prompt = toks[:6]
    assert cli.main(["generate", "--model", str(tmp_path), "--dtype", "float32", "--new-tokens", "5", "--prompt", ",".join(map(str, prompt))]) == 0
    line = json.loads(capsys.readouterr().out.strip().split("\n")[-1])
    assert line["tokens"] == oracle_greedy(cfg, w, prompt, 11)


def test_what_the_decoder_cannot_be_is_refused():
    import fandhe_ai_amd as fa
    cap = fa.models.Capacity(64, 1)
    bad = [left(heads=5), left(rot=22), left(rot=5), right(decay=[0.5, 1.5, 0.1]), right(decay=[0.5, -0.1, 0.1]), left_2(rot=30), right_2(heads=5),
           right_2(conv=0), right_2(conv=17), left_2(scaling=(2.0, 3.0, 1.0, 40))]
    for layer in bad:
        cfg = lc.bubetar([layer])
        with pytest.raises(fa.InvalidArgument):
            fa.models.build_layered(ops(), cfg, "bfloat16", cap, lc.shapes(cfg))
    for layer in (right(dim=300), right_2(vdim=1100)):
        cfg = lc.bubetar([layer])
        with pytest.raises(fa.Unsupported):
            fa.models.build_layered(ops(), cfg, "bfloat16", cap, lc.shapes(cfg))


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_any_two_mixers_stand_side_by_side(dtype):
    """Latent attention beside the delta rule with a decay per head, and two attentions, in a pre-norm stack with layer scales:
    the oracle's pieces put together."""
    import fandhe_ai_amd as fa
    from fandhe_ai_amd import capi
    D, V, T, eps = 64, 40, 70, 1e-5
    rng = np.random.default_rng(5)
    d, l, a = lc.delta(dim=16, vdim=16)["mixer"], lc.latent()["mixer"], lc.gated_left(4, 2, 16, 12, 8)
    delta = dict(mixer=capi.MIXER_DELTA, heads=d["heads"], kv_heads=d["kv_heads"], dim=16, vdim=16, conv=d["conv"], kv_from=-1)
    latent = dict(mixer=capi.MIXER_LATENT_ATTENTION, heads=l["heads"], dim=l["dim"], vdim=l["vdim"], q_rank=l["q_rank"], kv_rank=l["kv_rank"], rot_dim=l["rot_dim"],
                  window=13, scale=l["scale"], rot_base=1e4, kv_from=-1)
    gated = dict(mixer=capi.MIXER_ATTENTION, attention=capi.ATTENTION_HEAD_NORM | capi.ATTENTION_GATE, heads=4, kv_heads=2, dim=16, vdim=12, scale=a["scale"],
                 rot_dim=8, rot_base=3000.0, rot_interleaved=1, kv_from=-1)
    bare = dict(mixer=capi.MIXER_ATTENTION, heads=3, kv_heads=1, dim=8, vdim=20, scale=0.4, kv_from=-1)
    layers = [dict(latent, right=delta, left_scale=1.2, right_scale=0.7), dict(gated, right=bare, left_scale=-0.6, right_scale=1.1)]
    dec = fa.LayeredDecoder(ops(), D, V, layers, eps, 9.0, 8, 8, 1, dtype=fa.models.DTYPES[dtype])
    assert dec.state_slots == 1
    w = {}
    for n, s in dec.tensors().items():
        x = rng.normal(size=s) * (1.0 if len(s) == 1 or n == "embed" or n.endswith("conv") else s[1] ** -0.5)
        w[n] = lc.bf16_round((x - 1.0 if n.endswith(("A_log", "dt_bias")) else x).astype(np.float32))
        dec.set_tensor(n, w[n])
    w = {n: x.astype(np.float64) for n, x in w.items()}
    toks = [int(t) for t in rng.integers(0, V, T)]
    x = w["embed"][toks]
    h = oracle.layer_norm(x, w["l0.norm1"], eps)
    y = 1.2 * oracle.latent_mixer(h, oracle.latent_rows(h, w, "l0.mix.left.", l, eps), w, "l0.mix.left.", l, eps) + 0.7 * oracle.delta_mixer(h, w, "l0.mix.right.", d, eps)
    x = x + y * w["l0.ls1"]
    h = oracle.layer_norm(x, w["l1.norm1"], eps)
    q, k, v = ((h @ w["l1.mix.right." + n].T).reshape(T, g, -1) for n, g in (("q", 3), ("k", 1), ("v", 1)))
    y = -0.6 * oracle.gated_attention_mixer(h, w, "l1.mix.left.", a, eps) + 1.1 * (oracle.grouped_attention(q, k, v, 0.4).reshape(T, -1) @ w["l1.mix.right.o"].T)
    x = x + y * w["l1.ls1"]
    want = oracle.softcap(oracle.layer_norm(x, w["final.norm"], eps) @ w["head"].T, 9.0)
    assert lc.error(whole(dec, toks), want) < tolerance(dtype)
    assert lc.error(portions_of(dec, toks, (41,) + (1,) * 29), want) < tolerance(dtype)
    dec.close()
