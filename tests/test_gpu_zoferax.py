"""Zoferax models on the device against the float64 oracle (oracle/layered.py): grouped-query attention with normed
projections and shared caches, sparse experts, norms on the sublayers' outputs, additive positions; prompts, decoding,
portions, mixed batches, reuse of pages, far and hidden keys, and generation through the framework's own entry points."""
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


def compare(got, want, sure, dtype, what=None):
    """All positions in f32; in bf16 those whose experts are no close calls."""
    keep = np.ones(len(want), bool) if dtype == "float32" else sure
    assert keep.sum() >= 0.2 * len(want), "too few decided positions"
    assert lc.error(np.asarray(got)[keep], want[keep]) < tolerance(dtype), what


MECHANISMS = {
    "attention": [lc.attention()],
    "attention, a key head per query head": [lc.attention(heads=3, kv_heads=3, dim=16, vdim=16)],
    "attention, one key head": [lc.attention(heads=5, kv_heads=1, dim=9, vdim=7)],
    "attention, one head of one dim": [lc.attention(heads=1, kv_heads=1, dim=1, vdim=1, scale=0.7)],
    "attention 64 64": [lc.attention(heads=8, kv_heads=2, dim=64, vdim=64)],
    "attention 64 128": [lc.attention(heads=4, kv_heads=2, dim=48, vdim=128)],
    "attention 64 256": [lc.attention(heads=2, kv_heads=1, dim=64, vdim=200)],
    "attention 128 64": [lc.attention(heads=8, kv_heads=4, dim=128, vdim=40)],
    "attention 128 128": [lc.attention(heads=4, kv_heads=1, dim=128, vdim=128)],
    "attention 128 256": [lc.attention(heads=2, kv_heads=2, dim=100, vdim=132)],
    "attention 256 64": [lc.attention(heads=2, kv_heads=1, dim=256, vdim=64)],
    "attention 256 128": [lc.attention(heads=3, kv_heads=1, dim=130, vdim=96)],
    "attention 256 256": [lc.attention(heads=4, kv_heads=2, dim=192, vdim=256)],
    "attention beyond the matrix-core sizes": [lc.attention(heads=2, kv_heads=1, dim=300, vdim=260)],
    "attention, twenty query heads a key head": [lc.attention(heads=40, kv_heads=2, dim=8, vdim=12)],
    "attention, seventy query heads a key head": [lc.attention(heads=70, kv_heads=1, dim=16, vdim=8)],
    "negative scale": [lc.attention(scale=-0.4)],
    "shared cache": [lc.attention(), lc.attention(kv_from=0, scale=0.3), lc.attention(heads=3, kv_heads=1, dim=12, vdim=20),
                     lc.attention(heads=4, kv_from=0, scale=0.6), lc.attention(heads=5, kv_heads=1, dim=12, vdim=20, kv_from=2)],
    "experts": [lc.attention(mlp=lc.experts())],
    "one expert": [lc.attention(mlp=lc.experts(1, 1, 30))],
    "one of many experts": [lc.attention(mlp=lc.experts(20, 1, 17))],
    "all experts": [lc.attention(mlp=lc.experts(4, 4, 16))],
    "sixty of seventy experts": [lc.attention(mlp=lc.experts(70, 60, 8))],
    "two hundred experts": [lc.attention(mlp=lc.experts(200, 3, 9))],
    "all": [lc.attention(mlp=lc.experts()), lc.attention(heads=4, kv_heads=4, dim=32, vdim=32), lc.attention(kv_from=0, mlp=lc.experts(9, 3, 64)),
            lc.attention(heads=4, kv_heads=4, dim=32, vdim=32, kv_from=1, scale=0.1, mlp=lc.experts(3, 1, 50))],
}


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", sorted(MECHANISMS))
def test_mechanism_prompt_then_decode(name, dtype):
    """A prompt in one pass, every position's logits; then the same tokens with the last ones decoded one by one."""
    cfg = lc.zoferax(MECHANISMS[name])
    w = lc.weights(cfg, 11)
    toks = lc.tokens(cfg, 75, 3)
    want, sure = lc.decided(cfg, w, toks)
    dec = lc.make_decoder(ops(), cfg, w, dtype)
    compare(whole(dec, toks), want, sure, dtype)
    dec.set_sequences(tables_of(dec, 1), [0])
    got = [dec.forward([toks[:37]], [[36]])]
    for t in toks[37:]:
        got.append(dec.forward([[t]], [[0]]))
    compare(np.concatenate(got), want[36:], sure[36:], dtype)
    dec.close()


FORMS = {"attention plain": (33, 1), "attention few rows": (33, 2), "attention many rows": (33, 3), "attention, keys split further": (34, 8),
         "experts streamed": (29, 4), "experts in tiles": (29, 5), "experts in large tiles": (29, 6), "routed with the norm": (35, 1), "routed apart": (35, 2)}
FORM_LAYERS = {
    "all": MECHANISMS["all"],
    "large sizes": [lc.attention(heads=12, kv_heads=3, dim=128, vdim=128, mlp=lc.experts(6, 2, 272)), lc.attention(heads=12, kv_heads=3, dim=128, vdim=128, kv_from=0)],
    "wide heads": [lc.attention(heads=6, kv_heads=2, dim=200, vdim=160, mlp=lc.experts(40, 5, 33))],
}


@pytest.mark.parametrize("form", sorted(FORMS))
@pytest.mark.parametrize("name", sorted(FORM_LAYERS))
def test_every_kernel_form_gives_the_oracles_logits(name, form, tune):
    """bf16: prompts longer than a tile, portions behind cached tokens, and decoding, on every form of the kernels."""
    tune(*FORMS[form])
    cfg = lc.zoferax(FORM_LAYERS[name], width=256)
    w = lc.weights(cfg, 23)
    toks = lc.tokens(cfg, 700, 3)
    want, sure = lc.decided(cfg, w, toks)
    dec = lc.make_decoder(ops(), cfg, w, "bfloat16", max_tokens=1024)
    compare(whole(dec, toks), want, sure, "bfloat16")
    dec.set_sequences(tables_of(dec, 1), [0])
    got = [dec.forward([toks[:45]], [list(range(45))]), dec.forward([toks[45:600]], [list(range(555))]), dec.forward([toks[600:617]], [list(range(17))])]
    got += [dec.forward([[t]], [[0]]) for t in toks[617:650]]
    compare(np.concatenate(got), want[:650], sure[:650], "bfloat16")
    dec.close()


def test_residual_stream_after_every_layer():
    cfg = lc.zoferax(MECHANISMS["all"] + [lc.attention(heads=2, kv_heads=1)])
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


@pytest.mark.parametrize("width,vocab,block_size", [(64, 96, 16), (129, 50, 64), (320, 1000, 1), (1500, 40, 256)])
def test_other_widths_vocabularies_and_pages(width, vocab, block_size):
    cfg = lc.zoferax(MECHANISMS["all"], width=width, vocab=vocab, eps=3e-4, scale=0.2)
    w = lc.weights(cfg, 4)
    toks = lc.tokens(cfg, 80, 4)
    want, sure = lc.decided(cfg, w, toks)
    for dtype, as_bf16 in (("float32", True), ("float32", False), ("bfloat16", True)):
        dec = lc.make_decoder(ops(), cfg, w, dtype, as_bf16=as_bf16, block_size=block_size)
        compare(whole(dec, toks), want, sure, dtype)
        dec.close()


def test_positions_reach_the_model_only_through_the_embedding():
    """The additive positions far along, alone: no attention output, so a position's logits are its own token's."""
    cfg = lc.zoferax([lc.attention(heads=1, kv_heads=1, dim=4, vdim=4)], width=50, vocab=20, scale=0.01)
    w = lc.weights(cfg, 6)
    for n in ("l0.mix.v", "l0.mix.v.b"):
        w[n][:] = 0.0
    toks = [3] * 3000
    want = oracle.forward(cfg, w, toks)
    dec = lc.make_decoder(ops(), cfg, w, max_tokens=3008)
    assert lc.error(whole(dec, toks), want) < F32_TOL
    assert lc.error(want[1:], want[:-1]) > 100 * F32_TOL
    dec.close()


@pytest.mark.parametrize("use_graph", [False, True])
def test_steps_continue_a_prompt_pass(use_graph):
    cfg = lc.zoferax(MECHANISMS["all"])
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
    cfg = lc.zoferax(MECHANISMS["all"])
    w = lc.weights(cfg, 8)
    toks = lc.tokens(cfg, 230, 8)
    want, sure = lc.decided(cfg, w, toks)
    dec = lc.make_decoder(ops(), cfg, w, dtype)
    compare(whole(dec, toks), want, sure, dtype)
    for sizes in ((2,), (3, 2), (16,), (17, 15), (64,), (65, 63, 2), (7, 128), (100, 1, 1, 2)):
        dec.set_sequences(tables_of(dec, 1), [0])
        got, at, i = [], 0, 0
        while at < len(toks):
            n = min(sizes[i % len(sizes)], len(toks) - at)
            got.append(dec.forward([toks[at:at + n]], [list(range(n))]))
            at, i = at + n, i + 1
        compare(np.concatenate(got), want, sure, dtype, sizes)
    dec.close()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_mixed_batches_match_each_request_alone(dtype):
    """Portions of some beside single tokens of others, rows changing places, requests left out of steps."""
    cfg = lc.zoferax(MECHANISMS["all"])
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


def test_freed_pages_carry_nothing_over():
    """A pool of five pages: every later request runs on what earlier ones left behind, in another order."""
    cfg = lc.zoferax(MECHANISMS["all"])
    w = lc.weights(cfg, 10)
    dec = lc.make_decoder(ops(), cfg, w, max_tokens=80, max_batch=2)
    from fandhe_ai_amd.scheduler import PortionBatcher
    b = PortionBatcher(dec)
    for i, n in enumerate((70, 3, 40, 80, 1, 33)):
        toks = lc.tokens(cfg, n, 50 + i)
        first = n // 2 + 1
        got = b.feed([(i, toks[:first], list(range(first)))])
        for t in toks[first:]:
            got = np.concatenate([got, b.feed([(i, [t], [0])])])
        assert lc.error(got, oracle.forward(cfg, w, toks)) < F32_TOL, i
        b.release(i)
        if i % 2:
            b.feed([("takes a page %d" % i, [1], [])])
            b.release("takes a page %d" % i)
    assert b.free_pages() == 5
    dec.close()


def standing_out(heads, kv_heads, dim, vdim, n, at):
    """A model whose queries are all alike and in which one token's key wins every score that sees it by far: a position's
    attention output is that token's value exactly from the token on.  The sequence holds it at the places `at`."""
    cfg = lc.zoferax([lc.attention(heads, kv_heads, dim, vdim, scale=3.0), lc.attention(heads, kv_heads, dim, vdim, scale=3.0, kv_from=0)], width=96, vocab=40,
                     scale=1.0)
    w = lc.weights(cfg, 12)
    rng = np.random.default_rng(1)
    way = np.where(rng.random(dim) < 0.5, -1.0, 1.0)
    w["embed"][:, 70] = 3.0                                   # a slow channel of the additive positions: a steady value
    w["embed"][39, 70] = -3.0
    for i in (0, 1):
        w["l%d.mix.q" % i] = lc.bf16_round((0.02 * rng.normal(size=w["l%d.mix.q" % i].shape)).astype(np.float32))
        w["l%d.mix.q.b" % i] = lc.bf16_round(np.tile(way, heads).astype(np.float32))
        w["l%d.mix.q.norm" % i][:] = 1.0
    k = 0.05 * rng.normal(size=w["l0.mix.k"].shape)
    k[:, 70] = -np.tile(way, kv_heads)
    w["l0.mix.k"], w["l0.mix.k.norm"][:] = lc.bf16_round(k.astype(np.float32)), 1.0
    w["l0.mix.k.b"] = lc.bf16_round((0.1 * rng.normal(size=kv_heads * dim)).astype(np.float32))
    toks = [int(t) for t in rng.integers(0, 39, n)]
    for p in at:
        toks[p] = 39
    return cfg, w, toks


STANDING_OUT = [(4, 2, 16, 16, 400, (0,)), (4, 1, 16, 8, 420, (63, 300)), (6, 2, 64, 40, 330, (64,)), (2, 1, 128, 128, 700, (31, 511)), (4, 4, 200, 96, 150, (32, 33))]


@pytest.mark.parametrize("case", STANDING_OUT, ids=lambda c: "%d heads of %d %d" % (c[0], c[2], c[3]))
@pytest.mark.parametrize("dtype,form", [("float32", 0), ("bfloat16", 0), ("bfloat16", 1), ("bfloat16", 2), ("bfloat16", 3)])
def test_a_key_that_stands_out(dtype, case, form, tune):
    """The first token, tokens at page and tile borders, keys hundreds of tokens away: seen from their own position on and
    not before, in prompts, portions and decoding, in the layer itself and in one that uses its cache."""
    tune(33, form)
    cfg, w, toks = standing_out(*case)
    want = oracle.forward(cfg, w, toks)
    hidden = oracle.forward(cfg, w, [5 if t == 39 else t for t in toks])
    for p in (case[5][0], len(toks) - 1):                     # far beyond the tolerance: at its own place and at the far end
        assert lc.error(hidden[p:p + 1], want[p:p + 1]) > 0.3
    dec = lc.make_decoder(ops(), cfg, w, dtype, max_tokens=768)
    assert lc.error(whole(dec, toks), want) < tolerance(dtype)
    for cut in (1, case[5][-1] + 1, len(toks) - 40):
        dec.set_sequences(tables_of(dec, 1), [0])
        got = [dec.forward([toks[:cut]], [list(range(cut))])]
        mid = max(cut, len(toks) - 60)
        if mid > cut:
            got.append(dec.forward([toks[cut:mid]], [list(range(mid - cut))]))
        for t in toks[mid:]:
            got.append(dec.forward([[t]], [[0]]))
        assert lc.error(np.concatenate(got), want) < tolerance(dtype), cut
    dec.close()


def test_first_tokens():
    cfg = lc.zoferax(MECHANISMS["all"])
    w = lc.weights(cfg, 14)
    dec = lc.make_decoder(ops(), cfg, w)
    for n in range(1, 6):
        toks = lc.tokens(cfg, n, n)
        want = oracle.forward(cfg, w, toks)
        assert lc.error(whole(dec, toks), want) < F32_TOL
        dec.set_sequences(tables_of(dec, 1), [0])
        assert lc.error(np.concatenate([dec.forward([[t]], [[0]]) for t in toks]), want) < F32_TOL
    dec.close()


def test_a_whole_batch_of_one_token():
    """Every row takes the same experts: a group as long as the batch, the others empty; the groups' counters start over."""
    cfg = lc.zoferax([lc.attention(mlp=lc.experts(7, 2, 40)), lc.attention(kv_from=0, mlp=lc.experts(12, 1, 24))])
    w = lc.weights(cfg, 15)
    want, sure = lc.decided(cfg, w, [9, 9, 9])
    for dtype in ("float32", "bfloat16"):
        dec = lc.make_decoder(ops(), cfg, w, dtype, max_tokens=1600, max_batch=100)
        dec.set_sequences(tables_of(dec, 100), [0] * 100)
        for p in range(3):
            got = dec.forward([[9]] * 100, [[0]] * 100)
            assert not sure[p] and dtype != "float32" or lc.error(got, np.repeat(want[p:p + 1], 100, axis=0)) < tolerance(dtype), p
        dec.close()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_long_decoding_of_unequal_requests(dtype):
    """Three rows decoded together from graphs for 150 steps."""
    cfg = lc.zoferax(MECHANISMS["all"])
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
    """generate() and the batch scheduler against greedy decoding with the oracle; more requests than rows or pages."""
    from fandhe_ai_amd.scheduler import BatchScheduler, GenerateConfig, SamplingStrategy, SchedulerLimits, generate, generate_speculative
    cfg = lc.zoferax(MECHANISMS["all"])
    w = lc.weights(cfg, 16)
    prompts = [lc.tokens(cfg, n, 70 + n) for n in (3, 20, 9, 31, 1)]
    want = [oracle_greedy(cfg, w, p, len(p) + 12) for p in prompts]
    dec = lc.make_decoder(ops(), cfg, w, max_tokens=112, max_batch=3)
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
    # no recurrent state: a drafted continuation can be verified and cut back
    draft = lc.make_decoder(ops(), cfg, lc.weights(cfg, 17), max_tokens=112, max_batch=3)
    out, _, _ = generate_speculative(dec, draft, np.array(prompts[1]), GenerateConfig(len(want[1]), SamplingStrategy.Greedy()), 3)
    assert np.asarray(out).reshape(-1).tolist() == want[1]
    draft.close()
    dec.close()


def test_long_prompts_run_in_several_internal_passes(tune):
    cfg = lc.zoferax(MECHANISMS["all"])
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
    cfg = lc.zoferax(MECHANISMS["all"])
    w = lc.weights(cfg, 21)
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    typed = {n: fa.safetensors_io.TypedTensor("BF16", a.shape, (a.view(np.uint32) >> 16).astype(np.uint16)) for n, a in w.items()}
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
    for layers, error in (([lc.attention(heads=5, kv_heads=2)], fa.InvalidArgument), ([lc.attention(), lc.attention(kv_from=0, dim=24)], fa.InvalidArgument),
                          ([lc.attention(), lc.attention(kv_from=0), lc.attention(kv_from=1)], fa.InvalidArgument),
                          ([lc.attention(kv_from=0)], fa.InvalidArgument), ([lc.attention(mlp=lc.experts(4, 5))], fa.InvalidArgument),
                          ([lc.attention(mlp=lc.experts(300, 2))], fa.Unsupported)):
        with pytest.raises(error):
            fa.models.build_layered(ops(), lc.zoferax(layers), "bfloat16", cap)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_mechanisms_combine_with_those_of_other_designs(dtype):
    """Grouped-query attention without biases and norms in a pre-norm stack beside a dense feed-forward, and latent attention
    and a gated delta rule under norms at the output: residual streams of the two kinds of stack agree with the oracle's
    pieces put together."""
    import fandhe_ai_amd as fa
    from fandhe_ai_amd import capi
    D, V, T, eps = 64, 40, 50, 1e-5
    rng = np.random.default_rng(5)
    # pre-norm: attention + GLU
    layer = dict(mixer=capi.MIXER_ATTENTION, heads=4, kv_heads=2, dim=16, vdim=16, scale=0.5, kv_from=-1, d_ffn=48, ffn_limit=2.0, ffn_alpha=1.702)
    dec = fa.LayeredDecoder(ops(), D, V, [layer], eps, 9.0, 8, 8, 1, dtype=fa.models.DTYPES[dtype])
    w = {}
    for n, s in dec.tensors().items():
        a = rng.normal(size=s) * (1.0 if len(s) == 1 or n == "embed" else s[1] ** -0.5)
        w[n] = lc.bf16_round(a.astype(np.float32))
        dec.set_tensor(n, w[n])
    assert "l0.mix.q.b" not in w and "l0.mix.k.norm" not in w
    w = {n: a.astype(np.float64) for n, a in w.items()}
    toks = [int(t) for t in rng.integers(0, V, T)]
    x = w["embed"][toks]
    h = oracle.layer_norm(x, w["l0.norm1"], eps)
    q, k, v = ((h @ w["l0.mix." + n].T).reshape(T, -1, 16) for n in "qkv")
    x = x + (oracle.grouped_attention(q, k, v, 0.5).reshape(T, -1) @ w["l0.mix.o"].T) * w["l0.ls1"]
    x = x + oracle.clamped_glu(oracle.layer_norm(x, w["l0.norm2"], eps), w, "l0.mlp.", 2.0) * w["l0.ls2"]
    want = oracle.softcap(oracle.layer_norm(x, w["final.norm"], eps) @ w["head"].T, 9.0)
    assert lc.error(whole(dec, toks), want) < tolerance(dtype)
    dec.close()
    # norms at the output: delta, latent attention, dense feed-forward
    d, l = lc.delta(dim=16, vdim=16)["mixer"], lc.latent(mlp=None)["mixer"]
    layers = [dict(mixer=capi.MIXER_DELTA, heads=d["heads"], kv_heads=d["kv_heads"], dim=16, vdim=16, conv=d["conv"], kv_from=-1, d_ffn=40, ffn_limit=2.0, ffn_alpha=1.702),
              dict(mixer=capi.MIXER_LATENT_ATTENTION, heads=l["heads"], dim=l["dim"], vdim=l["vdim"], q_rank=l["q_rank"], kv_rank=l["kv_rank"], rot_dim=l["rot_dim"],
                   window=13, scale=l["scale"], rot_base=1e4, kv_from=-1)]
    dec = fa.LayeredDecoder(ops(), D, V, layers, eps, 0.0, 8, 8, 1, dtype=fa.models.DTYPES[dtype], norm=capi.NORM_OUTPUT, embed_scale=2.0)
    w = {}
    for n, s in dec.tensors().items():
        a = rng.normal(size=s) * (1.0 if len(s) == 1 or n == "embed" or n.endswith("conv") else s[1] ** -0.5)
        w[n] = lc.bf16_round((a - 1.0 if n.endswith(("A_log", "dt_bias")) else a).astype(np.float32))
        dec.set_tensor(n, w[n])
    w = {n: a.astype(np.float64) for n, a in w.items()}
    x = 2.0 * w["embed"][toks]
    x = x + oracle.rms_norm(oracle.delta_mixer(x, w, "l0.mix.", d, eps), w["l0.norm1"], eps)
    x = x + oracle.rms_norm(oracle.clamped_glu(x, w, "l0.mlp.", 2.0), w["l0.norm2"], eps)
    x = x + oracle.rms_norm(oracle.latent_mixer(x, oracle.latent_rows(x, w, "l1.mix.", l, eps), w, "l1.mix.", l, eps), w["l1.norm1"], eps)
    want = oracle.rms_norm(x, w["final.norm"], eps) @ w["head"].T
    assert lc.error(whole(dec, toks), want) < tolerance(dtype)
    dec.close()
