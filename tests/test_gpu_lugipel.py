"""Lugipel models on the device against the float64 oracle (oracle/layered.py): minimal gated recurrences, windowed attention
with sigmoid weights, distance biases, query temperature and gates per head, xIELU, experts chosen by scores in groups with identity
experts, RMS norms ahead of sublayers; prompts, decoding, portions, mixed batches, reuse of pages and state slots, far and
hidden keys, old states, and generation through the framework's own entry points."""
import copy

import numpy as np
import pytest

import layered_common as lc
from gpu_common import ops
from layered_common import oracle
from test_gpu_bubetar import portions_of
from test_gpu_layered import F32_TOL, oracle_greedy, step_logits, tables_of, whole

pytestmark = pytest.mark.gpu

BF16_TOL = 0.1
att, gru = lc.sigmoid_attention, lc.mingru


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


def compare(got, want, sure, dtype, what=None):
    """All positions in f32; in bf16 those whose experts are no close calls."""
    keep = np.ones(len(want), bool) if dtype == "float32" else sure
    assert keep.sum() >= 0.2 * len(want), "too few decided positions"
    assert lc.error(np.asarray(got)[keep], want[keep]) < tolerance(dtype), what


MECHANISMS = {
    "attention": [att()],
    "attention, a key head per query head": [att(heads=3, kv_heads=3, dim=16, vdim=16)],
    "attention, one key head": [att(heads=5, kv_heads=1, dim=9, vdim=7)],
    "attention, one head of one dim": [att(heads=1, kv_heads=1, dim=1, vdim=1, scale=0.7)],
    "attention 64 64": [att(heads=8, kv_heads=2, dim=64, vdim=64, window=37)],
    "attention 64 128": [att(heads=4, kv_heads=2, dim=48, vdim=128)],
    "attention 64 256": [att(heads=2, kv_heads=1, dim=64, vdim=200)],
    "attention 128 64": [att(heads=8, kv_heads=4, dim=128, vdim=40)],
    "attention 128 128": [att(heads=4, kv_heads=1, dim=128, vdim=128, window=32)],
    "attention 128 256": [att(heads=2, kv_heads=2, dim=100, vdim=132)],
    "attention 256 64": [att(heads=2, kv_heads=1, dim=256, vdim=64)],
    "attention 256 128": [att(heads=3, kv_heads=1, dim=130, vdim=96)],
    "attention 256 256": [att(heads=4, kv_heads=2, dim=192, vdim=256)],
    "attention beyond the matrix-core sizes": [att(heads=2, kv_heads=1, dim=300, vdim=260)],
    "attention, twenty query heads a key head": [att(heads=40, kv_heads=2, dim=8, vdim=12)],
    "attention, seventy query heads a key head": [att(heads=70, kv_heads=1, dim=16, vdim=8)],
    "window of one": [att(window=1)],
    "window longer than the sequence": [att(window=4096)],
    "a negative scale": [att(scale=-0.4)],
    "temperature at every position": [att(every=1, coef=0.4)],
    "no temperature": [att(coef=0.0), att(every=None)],
    "no window": [att(window=None), att(heads=2, kv_heads=1, dim=64, vdim=64, window=None, every=None)],
    "a negative temperature": [att(every=3, coef=-0.3)],
    "recurrence": [gru()],
    "recurrence of one channel": [gru(1)],
    "recurrence, odd width": [gru(67)],
    "recurrence, wider than the model": [gru(300)],
    "xIELU": [gru(mlp=lc.dense(52))],
    "experts": [gru(mlp=lc.scored())],
    "experts without groups": [gru(mlp=lc.scored(groups=None))],
    "experts without identity": [gru(mlp=lc.scored(8, 0, (4, 2), 3))],
    "one group kept": [gru(mlp=lc.scored(9, 3, (3, 1), 4))],
    "all groups kept": [gru(mlp=lc.scored(6, 2, (4, 4), 5))],
    "a group per expert": [gru(mlp=lc.scored(6, 2, (8, 3), 3))],
    "all experts": [gru(mlp=lc.scored(4, 2, None, 6, 16))],
    "one expert among identities": [gru(mlp=lc.scored(1, 5, (3, 2), 2))],
    "one expert alone": [gru(mlp=lc.scored(1, 0, None, 1))],
    "one of many": [gru(mlp=lc.scored(20, 4, (6, 2), 1, 17))],
    "sixty of eighty": [gru(mlp=lc.scored(70, 10, (8, 7), 60, 8))],
    "two hundred and forty outputs": [gru(mlp=lc.scored(200, 40, (120, 3), 5, 9))],
    "no feed-forward": [att(), gru(), att()],
    "all": [att(mlp=lc.dense()), gru(mlp=lc.scored()), att(heads=4, kv_heads=4, dim=32, vdim=32, window=9, mlp=lc.scored(5, 3, (4, 2), 3)), gru(30),
            att(heads=3, kv_heads=1, window=40, mlp=lc.scored(7, 0, None, 2, 64, 0.8)), gru(mlp=lc.dense(33))],
}


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", sorted(MECHANISMS))
def test_mechanism_prompt_then_decode(name, dtype):
    """A prompt in one pass, every position's logits; then the same tokens with the last ones decoded one by one."""
    cfg = lc.lugipel(MECHANISMS[name])
    w = lc.weights(cfg, 11)
    toks = lc.tokens(cfg, 75, 3)
    want, sure = lc.decided(cfg, w, toks)
    dec = lc.make_decoder(ops(), cfg, w, dtype)
    compare(whole(dec, toks), want, sure, dtype)
    compare(portions_of(dec, toks, (37,) + (1,) * 38), want, sure, dtype)
    dec.close()


FORMS = {"attention plain": (33, 1), "attention few rows": (33, 2), "attention many rows": (33, 3), "attention, keys split further": (34, 8),
         "experts streamed": (29, 4), "experts in tiles": (29, 5), "experts in large tiles": (29, 6), "routed with the norm": (35, 1), "routed apart": (35, 2),
         "scan of 8 lanes": (36, 8), "scan of 16 lanes": (36, 16)}
FORM_LAYERS = {
    "all": MECHANISMS["all"],
    "large sizes": [att(heads=12, kv_heads=3, dim=128, vdim=128, window=600, mlp=lc.scored(4, 2, (3, 2), 2, 272)), gru(260, mlp=lc.dense(520))],
    "wide heads": [att(heads=6, kv_heads=2, dim=200, vdim=160, window=90, mlp=lc.scored(38, 10, (6, 3), 5, 33))],
}


@pytest.mark.parametrize("form", sorted(FORMS))
@pytest.mark.parametrize("name", sorted(FORM_LAYERS))
def test_every_kernel_form_gives_the_oracles_logits(name, form, tune):
    """bf16: prompts longer than a tile, portions behind cached tokens, and decoding, on every form of the kernels."""
    tune(*FORMS[form])
    cfg = lc.lugipel(FORM_LAYERS[name], width=256)
    w = lc.weights(cfg, 23)
    toks = lc.tokens(cfg, 700, 3)
    want, sure = lc.decided(cfg, w, toks)
    dec = lc.make_decoder(ops(), cfg, w, "bfloat16", max_tokens=1024)
    compare(whole(dec, toks), want, sure, "bfloat16")
    got = portions_of(dec, toks[:650], (45, 555, 17) + (1,) * 33)
    compare(got, want[:650], sure[:650], "bfloat16")
    dec.close()


def test_residual_stream_after_every_layer():
    cfg = lc.lugipel(MECHANISMS["all"] + [att()])
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


@pytest.mark.parametrize("width,vocab,block_size", [(64, 96, 16), (129, 50, 64), (320, 1000, 1), (1500, 40, 256), (4100, 30, 16)])
def test_other_widths_vocabularies_and_pages(width, vocab, block_size):
    cfg = lc.lugipel(MECHANISMS["all"], width=width, vocab=vocab, eps=3e-4, scale=0.2)
    w = lc.weights(cfg, 4)
    toks = lc.tokens(cfg, 80, 4)
    want, sure = lc.decided(cfg, w, toks)
    for dtype, as_bf16 in (("float32", True), ("float32", False), ("bfloat16", True)):
        dec = lc.make_decoder(ops(), cfg, w, dtype, as_bf16=as_bf16, block_size=block_size)
        compare(whole(dec, toks), want, sure, dtype)
        dec.close()


@pytest.mark.parametrize("use_graph", [False, True])
def test_steps_continue_a_prompt_pass(use_graph):
    cfg = lc.lugipel(MECHANISMS["all"])
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
    cfg = lc.lugipel(MECHANISMS["all"])
    w = lc.weights(cfg, 8)
    toks = lc.tokens(cfg, 300, 8)
    want, sure = lc.decided(cfg, w, toks)
    dec = lc.make_decoder(ops(), cfg, w, dtype)
    compare(whole(dec, toks), want, sure, dtype)
    for sizes in ((2,), (3, 2), (5,), (16,), (17, 15), (64,), (65, 63, 2), (127, 2), (128,), (129, 1), (100, 1, 1, 2), (297, 2)):
        compare(portions_of(dec, toks, sizes), want, sure, dtype, sizes)
    dec.close()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_mixed_batches_match_each_request_alone(dtype):
    """Portions of some beside single tokens of others, rows changing places, requests left out of steps."""
    cfg = lc.lugipel(MECHANISMS["all"])
    w = lc.weights(cfg, 9)
    reqs = {r: lc.tokens(cfg, n, 20 + i) for i, (r, n) in enumerate((("a", 260), ("b", 33), ("c", 90), ("d", 5)))}
    ref = {r: lc.decided(cfg, w, t) for r, t in reqs.items()}
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
    for r in reqs:
        keep = np.ones(len(reqs[r]), bool) if dtype == "float32" else ref[r][1]
        assert lc.error(np.concatenate(got[r])[keep], ref[r][0][keep]) < tolerance(dtype), r
    dec.close()


def test_freed_pages_and_slots_carry_nothing_over():
    """A pool of five pages and two states: every later request runs on what earlier ones left behind, in another order."""
    cfg = lc.lugipel(MECHANISMS["all"])
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


def steady_model(layer, width=96):
    """One layer, and two channels of the residual that hardly depend on the position: 94 the same for every token, 92 with
    another sign for one of them."""
    cfg = lc.lugipel([layer], width=width, vocab=40, eps=1e-6, scale=1.0)
    w = lc.weights(cfg, 12)
    w["embed"][:, width - 4], w["embed"][:, width - 2] = 5.0, 5.0
    w["embed"][SPECIAL, width - 4] = -5.0
    w["l0.norm1"][:] = 1.0
    return cfg, w


def standing_out(heads, kv_heads, dim, vdim, window, n, at):
    """All queries alike, and one token whose key is the only one with a weight to speak of; the sequence holds it at the
    places `at`.  Heads with small slopes see it from far, those with large ones from near."""
    cfg, w = steady_model(att(heads, kv_heads, dim, vdim, window, 24.0 / dim, 0.1, 64))
    rng = np.random.default_rng(1)
    way = np.where(rng.random(dim) < 0.5, -1.0, 1.0)
    q, k = 0.02 * rng.normal(size=w["l0.mix.q"].shape), 0.02 * rng.normal(size=w["l0.mix.k"].shape)
    q[:, 94], k[:, 92] = np.tile(way, heads), -np.tile(way, kv_heads)
    w["l0.mix.q"], w["l0.mix.k"] = lc.bf16_round(q.astype(np.float32)), lc.bf16_round(k.astype(np.float32))
    w["l0.mix.q.norm"][:] = w["l0.mix.k.norm"][:] = 1.0
    w["l0.mix.pb"][:] = lc.bf16_round(rng.uniform(-1.0, 1.0, heads).astype(np.float32))
    w["l0.mix.o"] = w["l0.mix.o"] * 4.0
    toks = [int(t) for t in rng.integers(0, SPECIAL, n)]
    for p in at:
        toks[p] = SPECIAL
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


FAR = {"64, the first token": (4, 2, 16, 16, 1000, 400, (0,)), "64, page and tile borders": (4, 1, 16, 8, 600, 420, (63, 300)), "64": (6, 2, 64, 40, 500, 330, (64,)),
       "128": (2, 1, 128, 128, 700, 640, (31, 511)), "256": (4, 4, 200, 96, 300, 150, (32, 33))}
EVERY_FORM = pytest.mark.parametrize("dtype,form", [("float32", 0), ("bfloat16", 0), ("bfloat16", 1), ("bfloat16", 2), ("bfloat16", 3)])


@EVERY_FORM
@pytest.mark.parametrize("name", sorted(FAR))
def test_a_far_key_that_stands_out(name, dtype, form, tune):
    """Seen from its own position to the end, hundreds of tokens on, in prompts, portions and decoding."""
    tune(33, form)
    case = FAR[name]
    cfg, w, toks = standing_out(*case)
    want, hidden = oracle.forward(cfg, w, toks), oracle.forward(cfg, w, [5 if t == SPECIAL else t for t in toks])
    for p in (case[-1][0], len(toks) - 1):                    # far beyond the tolerance: at its own place and at the far end
        assert lc.error(hidden[p:p + 1], want[p:p + 1]) > 0.2, p
    check_standing_out(cfg, w, toks, dtype, (1, case[-1][-1] + 1, len(toks) - 40))


@EVERY_FORM
@pytest.mark.parametrize("dim,share,window", [(16, 2, 1), (16, 1, 16), (40, 3, 17), (128, 1, 33), (128, 4, 150), (200, 2, 64)])
def test_window_edges(dim, share, window, dtype, form, tune):
    """The key that stands out shows exactly as long as the window holds it."""
    tune(33, form)
    cfg, w, toks = standing_out(2 * share, 2, dim, 20, window, 3 * window + 40, (0, 15, 16, window + 20))
    want = oracle.forward(cfg, w, toks)
    for off in (-1, 1):                                       # a window one off would be seen, far beyond the tolerance
        if window + off < 1:
            continue
        wrong = copy.deepcopy(cfg)
        wrong["layers"][0]["mixer"]["mask"]["size"] = window + off
        assert lc.error(oracle.forward(wrong, w, toks), want) > 0.3
    check_standing_out(cfg, w, toks, dtype, (1, window, window + 21))


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_biases_from_no_key_to_every_key(dtype):
    """Heads that see nothing, heads that sum every value alike, and those in between."""
    for window in (3, 500):
        cfg = lc.lugipel([att(6, 3, 20, 16, window)])
        w = lc.weights(cfg, 31)
        w["l0.mix.pb"][:] = [-100.0, -6.0, 0.0, 2.5, 9.0, 200.0]
        toks = lc.tokens(cfg, 330, 31)
        want = oracle.forward(cfg, w, toks)
        dec = lc.make_decoder(ops(), cfg, w, dtype)
        assert lc.error(whole(dec, toks), want) < tolerance(dtype)
        assert lc.error(portions_of(dec, toks, (200, 90) + (1,) * 40), want) < tolerance(dtype)
        dec.close()


@pytest.mark.parametrize("width", [48, 131])
def test_what_was_written_long_ago_is_read_back_from_the_state(width):
    """One token writes everything, the others next to nothing: its candidate is read hundreds of tokens on, through portions
    and through decoding, until the token comes again."""
    cfg, w = steady_model(gru(width))
    w["l0.mix.z"][:, 92] = -8.0
    w["l0.mix.z.b"][:] = -9.0
    n = 420
    toks = [t % SPECIAL for t in lc.tokens(cfg, n, 1)]
    toks[3] = SPECIAL
    want = oracle.forward(cfg, w, toks)
    other = oracle.forward(cfg, dict(w, **{"l0.mix.x.b": np.roll(w["l0.mix.x.b"], 1)}), toks)
    for p in (3, 5, n - 1):
        assert lc.error(other[p:p + 1], want[p:p + 1]) > 500 * F32_TOL
    dec = lc.make_decoder(ops(), cfg, w)
    assert lc.error(whole(dec, toks), want) < F32_TOL
    assert lc.error(portions_of(dec, toks, (150, 35, 2, 128, 35, 35) + (1,) * 40), want) < F32_TOL
    toks[260] = SPECIAL
    assert lc.error(portions_of(dec, toks, (3, 130) + (1,) * 40), oracle.forward(cfg, w, toks)) < F32_TOL
    dec.close()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_gates_from_closed_to_open(dtype, tune):
    """Channels that never write beside channels that keep nothing; candidates on both sides of zero."""
    cfg = lc.lugipel([gru(64), gru(90)])
    w = lc.weights(cfg, 14)
    rng = np.random.default_rng(14)
    for i in (0, 1):
        w["l%d.mix.z.b" % i][:] = lc.bf16_round(rng.uniform(-30.0, 30.0, w["l%d.mix.z.b" % i].shape).astype(np.float32))
        w["l%d.mix.x.b" % i][:] = lc.bf16_round(rng.uniform(-8.0, 8.0, w["l%d.mix.x.b" % i].shape).astype(np.float32))
    toks = lc.tokens(cfg, 300, 14)
    want = oracle.forward(cfg, w, toks)
    dec = lc.make_decoder(ops(), cfg, w, dtype)
    for lanes in (8, 16):
        tune(36, lanes)
        for sizes in ((300,), (130, 17), (12, 11), (1,)):
            assert lc.error(portions_of(dec, toks, sizes), want) < tolerance(dtype), sizes
    dec.close()


def test_first_tokens():
    cfg = lc.lugipel(MECHANISMS["all"])
    w = lc.weights(cfg, 14)
    dec = lc.make_decoder(ops(), cfg, w)
    for n in range(1, 6):
        toks = lc.tokens(cfg, n, n)
        want = oracle.forward(cfg, w, toks)
        assert lc.error(whole(dec, toks), want) < F32_TOL
        assert lc.error(portions_of(dec, toks, (1,)), want) < F32_TOL
    dec.close()


def test_positions_far_along():
    """Additive positions and the temperature thousands of tokens on."""
    cfg = lc.lugipel([att(2, 1, 8, 8, 20, 0.5, 0.5, 100)], width=50, vocab=20, scale=0.05)
    w = lc.weights(cfg, 6)
    toks = lc.tokens(cfg, 3000, 2)
    want = oracle.forward(cfg, w, toks)
    flat = copy.deepcopy(cfg)
    flat["layers"][0]["mixer"]["q_temp"]["every"] = 101
    assert lc.error(oracle.forward(flat, w, toks)[-100:], want[-100:]) > 5 * F32_TOL
    dec = lc.make_decoder(ops(), cfg, w, max_tokens=3008)
    assert lc.error(whole(dec, toks), want) < F32_TOL
    dec.close()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("identity_first", [False, True])
def test_a_whole_batch_takes_the_same_experts(identity_first, dtype):
    """A list as long as the batch, the others empty; nothing but identity experts, no list at all; the lists' counters start
    over."""
    cfg = lc.lugipel([gru(mlp=lc.scored(6, 6, (4, 2), 4, 40)), att(mlp=lc.scored(9, 3, None, 2, 24))])
    w = lc.weights(cfg, 15)
    for p in ("l0.mlp.correction", "l1.mlp.correction"):
        w[p][:] = 0.0
        w[p][-6 if p[1] == "0" else -3:] = 3.0 if identity_first else -3.0
    want, sure = lc.decided(cfg, w, [9, 9, 9])
    dec = lc.make_decoder(ops(), cfg, w, dtype, max_tokens=1600, max_batch=100)
    dec.set_sequences(tables_of(dec, 100), [0] * 100)
    for p in range(3):
        got = dec.forward([[9]] * 100, [[0]] * 100)
        assert not sure[p] and dtype != "float32" or lc.error(got, np.repeat(want[p:p + 1], 100, axis=0)) < tolerance(dtype), p
    dec.close()


@pytest.mark.parametrize("groups,keep", [(1, 1), (2, 1), (4, 2), (8, 5), (16, 3)])
def test_choice_of_experts_by_groups_with_negative_scores(groups, keep):
    """Choice scores below zero everywhere, so that an expert counted as zero would win; f32 and both of the bf16 routers."""
    cfg = lc.lugipel([gru(mlp=lc.scored(11, 5, (groups, keep), min(3, 16 // groups * keep), 20))])
    w = lc.weights(cfg, 16)
    rng = np.random.default_rng(groups)
    w["l0.mlp.correction"][:] = lc.bf16_round((-2.0 + 0.3 * rng.normal(size=16)).astype(np.float32))
    toks = lc.tokens(cfg, 150, 4)
    want, sure = lc.decided(cfg, w, toks)
    for dtype in ("float32", "bfloat16"):
        dec = lc.make_decoder(ops(), cfg, w, dtype)
        compare(whole(dec, toks), want, sure, dtype)
        compare(portions_of(dec, toks, (40, 1)), want, sure, dtype)
        dec.close()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_long_decoding_of_unequal_requests(dtype):
    """Three rows decoded together from graphs for 150 steps."""
    cfg = lc.lugipel(MECHANISMS["all"])
    w = lc.weights(cfg, 15)
    rows = [lc.tokens(cfg, n + 150, 60 + n) for n in (1, 18, 500)]
    dec = lc.make_decoder(ops(), cfg, w, dtype, max_tokens=2100)
    dec.set_sequences(tables_of(dec, 3), [0, 0, 0])
    dec.prefill_padded([r[:-150] for r in rows])
    ref = [lc.decided(cfg, w, r) for r in rows]
    got = [[] for _ in rows]
    for t in range(150):
        dec.set_tokens([r[len(r) - 150 + t] for r in rows])
        dec.step()
        for g, x in zip(got, dec.logits()):
            g.append(x)
    for g, (want, sure) in zip(got, ref):
        compare(g, want[-150:], sure[-150:], dtype)
    dec.close()


def test_greedy_generation_and_scheduler():
    """generate() and the batch scheduler against greedy decoding with the oracle; more requests than rows, pages or states."""
    from fandhe_ai_amd.scheduler import BatchScheduler, GenerateConfig, InvalidArgument, SamplingStrategy, SchedulerLimits, generate, generate_speculative
    cfg = lc.lugipel(MECHANISMS["all"])
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
    cfg = lc.lugipel(MECHANISMS["all"])
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
    import io
    import json
    import types
    import fandhe_ai_amd as fa
    from fandhe_ai_amd import __main__ as cli
    from fandhe_ai_amd import trace
    cfg = lc.lugipel(MECHANISMS["all"])
    w = lc.weights(cfg, 21)
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    typed = {n: fa.safetensors_io.TypedTensor("BF16", a.shape, (a.view(np.uint32) >> 16).astype(np.uint16)) for n, a in w.items()}
    typed["l3.norm2"] = typed["l3.norm1"]                     # of a feed-forward that the layer has not: passed over
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
    for layer in (att(heads=5), gru(0), gru(mlp=lc.scored(4, 0, None, 5)), gru(mlp=lc.scored(6, 3, (4, 2), 2)), gru(mlp=lc.scored(6, 3, (3, 1), 4)),
                  gru(mlp=lc.scored(6, 3, (3, 4), 2))):
        with pytest.raises(fa.InvalidArgument):
            fa.models.build_layered(ops(), lc.lugipel([layer]), "bfloat16", cap)
    for layer in (gru(mlp=lc.scored(250, 10, None, 2)), gru(mlp=lc.scored(0, 4, None, 2)), gru(mlp=lc.scored(80, 0, None, 70))):
        with pytest.raises(fa.Unsupported):
            fa.models.build_layered(ops(), lc.lugipel([layer]), "bfloat16", cap)


def random_model(dec, rng):
    w = {}
    for n, s in dec.tensors().items():
        a = rng.normal(size=s) * (1.0 if len(s) == 1 or n == "embed" or n.endswith("conv") else s[1] ** -0.5)
        w[n] = lc.bf16_round((a - 1.0 if n.endswith(("A_log", "dt_bias")) else a).astype(np.float32))
        dec.set_tensor(n, w[n])
    return {n: a.astype(np.float64) for n, a in w.items()}


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_mechanisms_combine_with_those_of_other_designs(dtype):
    """A minimal gated recurrence beside rotated attention and xIELU under layer norm and layer scale; softmax attention with
    distance biases and sigmoid attention over an earlier layer's cache under RMS norms ahead of sublayers, with experts chosen
    and weighted by their logits; scored experts with identity under norms at the output."""
    import fandhe_ai_amd as fa
    from fandhe_ai_amd import capi
    D, V, T, eps = 64, 40, 70, 1e-5
    rng = np.random.default_rng(5)
    toks = [int(t) for t in rng.integers(0, V, T)]
    silu_moe, relu_moe = {"router": {"experts": 5, "identity": 2, "top": 3, "scale": 1.3}}, {"router": {"experts": 6, "top": 2}}
    margins = []

    def check(dec, want):
        sure = np.min(margins + [np.full(T, np.inf)], axis=0) >= 0.05
        compare(whole(dec, toks), want, sure, dtype)
        compare(portions_of(dec, toks, (41,) + (1,) * 29), want, sure, dtype)
        dec.close()

    a = lc.gated_left(4, 2, 16, 12, 8)
    gated = dict(mixer=capi.MIXER_ATTENTION, attention=capi.ATTENTION_HEAD_NORM | capi.ATTENTION_GATE, heads=4, kv_heads=2, dim=16, vdim=12, scale=a["scale"],
                 rot_dim=8, rot_base=3000.0, rot_interleaved=1, kv_from=-1)
    mingru = dict(mixer=capi.MIXER_MINGRU, heads=1, dim=1, vdim=45, kv_from=-1)
    dec = fa.LayeredDecoder(ops(), D, V, [dict(gated, right=mingru, left_scale=0.8, right_scale=-1.2, d_ffn=50, glu=capi.FFN_XIELU)], eps, 9.0, 8, 8, 1,
                            dtype=fa.models.DTYPES[dtype])
    assert dec.state_slots == 1
    w = random_model(dec, rng)
    x = w["embed"][toks]
    h = oracle.layer_norm(x, w["l0.norm1"], eps)
    x = x + (0.8 * oracle.gated_attention_mixer(h, w, "l0.mix.left.", a, eps) - 1.2 * oracle.mingru_mixer(h, w, "l0.mix.right.")) * w["l0.ls1"]
    x = x + oracle.xielu_forward(oracle.layer_norm(x, w["l0.norm2"], eps), w, "l0.mlp.") * w["l0.ls2"]
    check(dec, oracle.softcap(oracle.layer_norm(x, w["final.norm"], eps) @ w["head"].T, 9.0))

    base = dict(mixer=capi.MIXER_ATTENTION, heads=4, kv_heads=2, dim=16, vdim=16, scale=0.4, kv_from=-1, distance=5.0)
    layers = [dict(base, window=20, d_ffn=24, experts=6, top=2), dict(base, attention=capi.ATTENTION_SIGMOID, kv_from=0, distance=0.0, d_ffn=40, glu=capi.GLU_SILU)]
    dec = fa.LayeredDecoder(ops(), D, V, layers, eps, 0.0, 8, 8, 1, dtype=fa.models.DTYPES[dtype], norm=capi.NORM_INPUT_RMS)
    assert dec.state_slots == 0
    w = random_model(dec, rng)
    x = w["embed"][toks]
    h = oracle.rms_norm(x, w["l0.norm1"], eps)
    q, k, v = ((h @ w["l0.mix." + n].T).reshape(T, -1, 16) for n in "qkv")
    o = np.empty_like(q)
    for t in range(T):
        j = np.arange(max(0, t - 19), t + 1)
        for n in range(4):
            e = np.exp(0.4 * k[j, n // 2] @ q[t, n] - 2.0 ** (-5.0 * (n + 1) / 4) * (t - j))
            o[t, n] = e @ v[j, n // 2] / e.sum()
    x = x + o.reshape(T, -1) @ w["l0.mix.o"].T
    x = x + oracle.sparse_experts(oracle.rms_norm(x, w["l0.norm2"], eps), w, "l0.mlp.", relu_moe, margins)
    h = oracle.rms_norm(x, w["l1.norm1"], eps)
    q = (h @ w["l1.mix.q"].T).reshape(T, 4, 16)
    x = x + oracle.sigmoid_attention(q, k, v, 0.4, None, np.zeros(4), w["l1.mix.pb"]).reshape(T, -1) @ w["l1.mix.o"].T
    x = x + oracle.silu_glu(oracle.rms_norm(x, w["l1.norm2"], eps), w, "l1.mlp.")
    check(dec, oracle.rms_norm(x, w["final.norm"], eps) @ w["head"].T)

    margins.clear()
    layers = [dict(mingru, d_ffn=24, experts=7, identity=2, top=3, glu=capi.GLU_SILU, route=capi.ROUTE_SCORED, route_scale=1.3)]
    dec = fa.LayeredDecoder(ops(), D, V, layers, eps, 0.0, 8, 8, 1, dtype=fa.models.DTYPES[dtype], norm=capi.NORM_OUTPUT)
    w = random_model(dec, rng)
    x = w["embed"][toks]
    x = x + oracle.rms_norm(oracle.mingru_mixer(x, w, "l0.mix."), w["l0.norm1"], eps)
    x = x + oracle.rms_norm(oracle.scored_experts(x, w, "l0.mlp.", silu_moe, margins), w["l0.norm2"], eps)
    check(dec, oracle.rms_norm(x, w["final.norm"], eps) @ w["head"].T)
