"""Layered decoders on the device against the float64 oracle (oracle/layered.py): every mechanism alone, prompts,
decoding, portions, mixed batches, reuse of pages and state slots, window edges, and generation through the framework's
own entry points."""
import numpy as np
import pytest

import layered_common as lc
from gpu_common import ops
from layered_common import oracle

pytestmark = pytest.mark.gpu

F32_TOL, BF16_TOL = 2e-4, 0.12


def stack_for(dtype):
    """Every mechanism, with fewer layers where each adds roundings."""
    return MECHANISMS["all"] if dtype == "float32" else [lc.latent(mlp=lc.glu()), lc.delta(heads=3, kv_heads=3), lc.latent(kv_from=0, window=25)]


@pytest.fixture(params=[("latent", 1), ("latent", 2), ("latent", 3), ("delta", 1)], ids=lambda p: "%s form %d" % p)
def form(request):
    """A kernel form other than the one chosen by shape: latent attention 1 plain, 2 absorbed, 3 expanded; delta 1 token by
    token."""
    from fandhe_ai_amd.capi import lib
    key = {"latent": 30, "delta": 31}[request.param[0]]
    assert lib.fa_set_tuning(key, request.param[1]) == 0
    yield request.param
    lib.fa_set_tuning(key, 0)


def tables_of(dec, rows):
    """Block tables that give row b the pages b, b + rows, ... (neighbouring pages belong to different rows)."""
    t = np.full((rows, dec.cfg.max_blocks_per_seq), 0xFFFFFFFF, dtype=np.uint32)
    n = dec.cfg.num_blocks // rows
    for b in range(rows):
        t[b, :n] = b + rows * np.arange(n)
    return t


def whole(dec, toks):
    dec.set_sequences(tables_of(dec, 1), [0])
    return dec.forward([toks], [list(range(len(toks)))])


MECHANISMS = {
    "delta": [lc.delta()],
    "delta one head group": [lc.delta(heads=2, kv_heads=2, dim=16, vdim=32, conv=3)],
    "delta one kv head, no convolution history": [lc.delta(heads=5, kv_heads=1, dim=9, vdim=7, conv=1)],
    "delta wide": [lc.delta(heads=2, kv_heads=1, dim=130, vdim=260, conv=2)],
    "delta 256": [lc.delta(heads=2, kv_heads=1, dim=256, vdim=48, conv=5)],
    "delta 128": [lc.delta(heads=4, kv_heads=2, dim=128, vdim=128, conv=4)],
    "delta with feed-forward": [lc.delta(mlp=lc.glu())],
    "latent": [lc.latent()],
    "latent aligned": [lc.latent(heads=16, dim=32, rot=32, vdim=32, q_rank=64, kv_rank=64, window=40)],
    "latent 512": [lc.latent(heads=20, dim=128, rot=64, vdim=128, q_rank=192, kv_rank=512, window=70)],
    "latent one head, tiny sizes": [lc.latent(heads=1, dim=1, rot=2, vdim=1, q_rank=3, kv_rank=5, window=4)],
    "latent window of one": [lc.latent(window=1)],
    "latent window longer than the sequence": [lc.latent(window=4096)],
    "latent shared cache": [lc.latent(window=9), lc.latent(heads=5, dim=8, vdim=12, q_rank=17, window=21, scale=0.3, kv_from=0)],
    "latent two rotations": [lc.latent(rot=4, base=100.0), lc.latent(rot=12, base=1e6)],
    "feed-forward": [lc.latent(mlp=lc.glu(ff=77, limit=0.8))],
    "all": [lc.latent(mlp=lc.glu()), lc.delta(), lc.delta(heads=3, kv_heads=3, mlp=lc.glu(33, 2.5)),
            lc.latent(kv_from=0, window=25, mlp=lc.glu(64)), lc.latent(kv_rank=60, window=8), lc.delta(conv=2), lc.latent(kv_from=4, kv_rank=60, heads=2)],
}


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", sorted(MECHANISMS))
def test_mechanism_prompt_then_decode(name, dtype):
    """A prompt in one pass, every position's logits; then the same tokens with the last ones decoded one by one."""
    cfg = lc.config(MECHANISMS[name])
    w = lc.weights(cfg, 11)
    toks = lc.tokens(cfg, 61, 3)
    want = oracle.forward(cfg, w, toks)
    dec = lc.make_decoder(ops(), cfg, w, dtype)
    tol = F32_TOL if dtype == "float32" else BF16_TOL
    assert lc.error(whole(dec, toks), want) < tol
    dec.set_sequences(tables_of(dec, 1), [0])
    got = [dec.forward([toks[:37]], [[36]])]
    for t in toks[37:]:
        got.append(dec.forward([[t]], [[0]]))
    assert lc.error(np.concatenate(got), want[36:]) < tol
    dec.close()


FORM_LAYERS = {
    "all": MECHANISMS["all"],
    "large sizes": [lc.latent(heads=20, dim=128, rot=64, vdim=128, q_rank=64, kv_rank=512, window=70), lc.delta(heads=2, kv_heads=1, dim=128, vdim=128)],
    "middle sizes": [lc.latent(heads=5, dim=70, rot=40, vdim=100, q_rank=64, kv_rank=200, window=33), lc.delta(heads=3, kv_heads=1, dim=40, vdim=72, conv=6)],
    "more than 32 heads": [lc.latent(heads=40, dim=16, rot=8, vdim=16, q_rank=32, kv_rank=32, window=300)],
}


@pytest.mark.parametrize("name", sorted(FORM_LAYERS))
def test_every_kernel_form_gives_the_oracles_logits(name, form):
    """bf16: whole prompts longer than a tile, portions behind cached tokens, and decoding, on every form of the kernels."""
    cfg = lc.config(FORM_LAYERS[name])
    w = lc.weights(cfg, 23)
    toks = lc.tokens(cfg, 290, 3)
    want = oracle.forward(cfg, w, toks)
    dec = lc.make_decoder(ops(), cfg, w, "bfloat16")
    tol = 0.2 if name == "all" else BF16_TOL               # roundings of seven layers
    assert lc.error(whole(dec, toks), want) < tol
    dec.set_sequences(tables_of(dec, 1), [0])
    got = [dec.forward([toks[:45]], [list(range(45))]), dec.forward([toks[45:200]], [list(range(155))]), dec.forward([toks[200:217]], [list(range(17))])]
    got += [dec.forward([[t]], [[0]]) for t in toks[217:250]]
    assert lc.error(np.concatenate(got), want[:250]) < tol
    dec.close()


def test_residual_stream_after_every_layer():
    cfg = lc.config(MECHANISMS["all"])
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


@pytest.mark.parametrize("width,vocab", [(64, 96), (129, 50), (320, 1000)])
def test_other_widths_and_vocabularies(width, vocab):
    cfg = lc.config(MECHANISMS["all"][:4], width=width, vocab=vocab, eps=3e-4, softcap=4.0)
    w = lc.weights(cfg, 4)
    toks = lc.tokens(cfg, 25, 4)
    want = oracle.forward(cfg, w, toks)
    for dtype, tol, as_bf16 in (("float32", F32_TOL, True), ("float32", F32_TOL, False), ("bfloat16", BF16_TOL, True)):
        dec = lc.make_decoder(ops(), cfg, w, dtype, as_bf16=as_bf16)
        assert lc.error(whole(dec, toks), want) < tol
        dec.close()


def step_logits(dec, toks, start, use_graph):
    out = []
    for t in toks[start:]:
        dec.set_tokens([t])
        dec.step(use_graph)
        out.append(dec.logits()[0])
    return np.array(out)


@pytest.mark.parametrize("use_graph", [False, True])
def test_steps_continue_a_prompt_pass(use_graph):
    """fa_decoder_prefill and fa_decoder_step (eager, and replayed from a graph) against one whole pass."""
    cfg = lc.config(MECHANISMS["all"])
    w = lc.weights(cfg, 7)
    toks = lc.tokens(cfg, 70, 7)
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
    cfg = lc.config(stack_for(dtype))
    w = lc.weights(cfg, 8)
    toks = lc.tokens(cfg, 230, 8)
    dec = lc.make_decoder(ops(), cfg, w, dtype)
    ref = whole(dec, toks)
    if dtype == "float32":
        assert lc.error(ref, oracle.forward(cfg, w, toks)) < F32_TOL
    for sizes in ((2,), (3, 2), (16,), (17, 15), (64,), (65, 63, 2), (7, 128), (100, 1, 1, 2)):
        dec.set_sequences(tables_of(dec, 1), [0])
        got, at, i = [], 0, 0
        while at < len(toks):
            n = min(sizes[i % len(sizes)], len(toks) - at)
            got.append(dec.forward([toks[at:at + n]], [list(range(n))]))
            at, i = at + n, i + 1
        assert lc.error(np.concatenate(got), ref) < (5e-5 if dtype == "float32" else BF16_TOL), sizes
    dec.close()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_mixed_batches_match_each_request_alone(dtype):
    """Portions of some beside single tokens of others, rows changing places, requests left out of steps."""
    cfg = lc.config(stack_for(dtype))
    w = lc.weights(cfg, 9)
    reqs = {r: lc.tokens(cfg, n, 20 + i) for i, (r, n) in enumerate((("a", 150), ("b", 33), ("c", 90), ("d", 5)))}
    dec = lc.make_decoder(ops(), cfg, w, dtype)
    ref = {r: whole(dec, t) for r, t in reqs.items()}
    rng = np.random.default_rng(3)
    from fandhe_ai_amd.scheduler import PortionBatcher
    b = PortionBatcher(dec)
    at = dict.fromkeys(reqs, 0)
    tol = 5e-5 if dtype == "float32" else BF16_TOL
    while any(at[r] < len(t) for r, t in reqs.items()):
        names = [r for r in reqs if at[r] < len(reqs[r]) and rng.random() < 0.8]
        rng.shuffle(names)
        entries = []
        for r in names:
            n = min(int(rng.choice([1, 1, 2, 3, 16, 40])), len(reqs[r]) - at[r])
            entries.append((r, reqs[r][at[r]:at[r] + n], list(range(n))))
        if not entries:
            continue
        want = np.concatenate([ref[r][at[r]:at[r] + len(t)] for r, t, _ in entries])
        assert lc.error(b.feed(entries), want) < tol, entries
        for r, t, _ in entries:
            at[r] += len(t)
    dec.close()


def test_freed_pages_and_slots_carry_nothing_over():
    """A pool of five pages and two slots: every later request runs on what an earlier one left behind."""
    cfg = lc.config(MECHANISMS["all"])
    w = lc.weights(cfg, 10)
    dec = lc.make_decoder(ops(), cfg, w, max_tokens=80, max_batch=2, state_slots=2)
    from fandhe_ai_amd.scheduler import PortionBatcher
    b = PortionBatcher(dec)
    for i, n in enumerate((70, 3, 40, 80, 1, 33)):
        toks = lc.tokens(cfg, n, 50 + i)
        got = b.feed([(i, toks[:n // 2 + 1], list(range(n // 2 + 1)))])
        if n > n // 2 + 1:
            rest = toks[n // 2 + 1:]
            got = np.concatenate([got, b.feed([(i, rest, list(range(len(rest))))])])
        assert lc.error(got, oracle.forward(cfg, w, toks)) < F32_TOL, i
        b.release(i)
        if i % 2:
            b.feed([("keeps a slot %d" % i, [1], [])])
            b.release("keeps a slot %d" % i)
    assert b.free_pages() == 5
    dec.close()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("kv_rank,window", [(44, 1), (44, 16), (64, 17), (64, 33), (96, 48), (512, 64)])
def test_window_edges_with_a_key_that_stands_out(dtype, kv_rank, window):
    window_edges(dtype, kv_rank, window)


@pytest.mark.parametrize("kv_rank,window", [(64, 17), (512, 64), (96, 150)])
def test_window_edges_on_every_kernel_form(kv_rank, window, form):
    window_edges("bfloat16", kv_rank, window)


def window_edges(dtype, kv_rank, window):
    """One token's key is made to win every score that sees it, so a position's output is that token's value exactly as
    long as the window holds it: the edge shows at full size, in prompts and decoded, across page borders."""
    cfg = lc.config([lc.latent(heads=4, dim=16, rot=4, vdim=16, q_rank=24, kv_rank=kv_rank, window=window, scale=3.0, base=1e9)], width=64, vocab=40)
    w = lc.weights(cfg, 12)
    rng = np.random.default_rng(1)
    # all queries alike (a constant direction of the residual), the special token's latent along it
    w["embed"][:, 0] = 3.0
    w["l0.mix.dq"] = lc.bf16_round(0.02 * rng.normal(size=w["l0.mix.dq"].shape))
    w["l0.mix.dq"][:, 0] = 1.0
    special = 39
    toks = [int(t) for t in rng.integers(0, 39, 3 * window + 40)]
    for at in (0, 15, 16, window + 20):
        toks[at] = special
    w["embed"][special] *= -1.0
    want = oracle.forward(cfg, w, toks)
    for off in (-1, 1):                                       # a window one off would be seen, far beyond the tolerance
        if window + off < 1:
            continue
        wrong = lc.config([dict(cfg["layers"][0], mixer=dict(cfg["layers"][0]["mixer"], mask={"size": window + off}))], width=64, vocab=40)
        assert lc.error(oracle.forward(wrong, w, toks), want) > 0.4
    tol = F32_TOL if dtype == "float32" else 0.15
    dec = lc.make_decoder(ops(), cfg, w, dtype)
    assert lc.error(whole(dec, toks), want) < tol
    for cut in (1, window, window + 21):
        dec.set_sequences(tables_of(dec, 1), [0])
        got = [dec.forward([toks[:cut]], [list(range(cut))])]
        for t in toks[cut:]:
            got.append(dec.forward([[t]], [[0]]))
        assert lc.error(np.concatenate(got), want) < tol, cut
    dec.close()


def test_a_far_write_is_read_back_from_the_recurrent_state():
    """Decays near one and one early token with a key of its own that the last tokens ask for: what was written hundreds
    of tokens ago must come back, through portions and through decoding."""
    cfg = lc.config([lc.delta(heads=2, kv_heads=1, dim=32, vdim=16, conv=2)], width=64, vocab=40)
    w = lc.weights(cfg, 13)
    w["l0.mix.A_log"][:] = -9.0
    n = 400
    toks = lc.tokens(cfg, n, 1)
    toks[3] = 39
    toks[-1] = 39
    want = oracle.forward(cfg, w, toks)
    other = list(toks)
    other[3] = 17
    assert lc.error(oracle.forward(cfg, w, other)[-1:], want[-1:]) > 100 * F32_TOL
    dec = lc.make_decoder(ops(), cfg, w)
    assert lc.error(whole(dec, toks), want) < F32_TOL
    dec.set_sequences(tables_of(dec, 1), [0])
    dec.forward([toks[:150]])
    for at in range(150, n - 40, 35):
        dec.forward([toks[at:min(at + 35, n - 40)]])
    got = np.concatenate([dec.forward([[t]], [[0]]) for t in toks[n - 40:]])
    assert lc.error(got, want[n - 40:]) < F32_TOL
    dec.close()


def test_first_tokens_and_strong_decay():
    """Sequences of one to five tokens (shorter than the convolution), decays down to nothing, full writes."""
    cfg = lc.config([lc.delta(conv=4), lc.latent(window=2), lc.delta(heads=2, kv_heads=1, conv=3)])
    w = lc.weights(cfg, 14)
    w["l0.mix.A_log"][:2] = 6.0
    w["l0.mix.dt_bias"][:2] = 8.0
    dec = lc.make_decoder(ops(), cfg, w)
    for n in range(1, 6):
        toks = lc.tokens(cfg, n, n)
        want = oracle.forward(cfg, w, toks)
        assert lc.error(whole(dec, toks), want) < F32_TOL
        dec.set_sequences(tables_of(dec, 1), [0])
        got = np.concatenate([dec.forward([[t]], [[0]]) for t in toks])
        assert lc.error(got, want) < F32_TOL
    dec.close()


def test_long_decoding_batch_of_unequal_requests():
    """Three rows decoded together from graphs for 150 steps, their windows and pages passing over decoded tokens."""
    cfg = lc.config(MECHANISMS["all"][:5])
    w = lc.weights(cfg, 15)
    rows = [lc.tokens(cfg, n + 150, 60 + n) for n in (1, 18, 50)]
    dec = lc.make_decoder(ops(), cfg, w, max_tokens=768)
    dec.set_sequences(tables_of(dec, 3), [0, 0, 0])
    dec.prefill_padded([r[:-150] for r in rows])
    want = [oracle.forward(cfg, w, r) for r in rows]
    assert lc.error(dec.logits(), np.array([x[-151] for x in want])) < F32_TOL
    for t in range(150):
        dec.set_tokens([r[len(r) - 150 + t] for r in rows])
        dec.step()
        if t % 7 == 0 or t == 149:
            assert lc.error(dec.logits(), np.array([x[len(x) - 150 + t] for x in want])) < F32_TOL, t
    dec.close()


def oracle_greedy(cfg, w, prompt, n):
    toks = list(prompt)
    while len(toks) < n:
        toks.append(int(oracle.forward(cfg, w, toks)[-1].argmax()))
    return toks


def test_greedy_generation_and_scheduler():
    """generate() and the batch scheduler against greedy decoding with the oracle; more requests than rows, slots or pages."""
    from fandhe_ai_amd.scheduler import BatchScheduler, GenerateConfig, SamplingStrategy, SchedulerLimits, generate
    cfg = lc.config(MECHANISMS["all"][:4])
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
    # sampled requests draw from their own generators: the same seeds give the same tokens alone and together
    strat = SamplingStrategy.Temperature(0.8)
    alone = [generate(dec, np.array(p), GenerateConfig(len(p) + 6, strat, 5 + i).clone()).tolist() for i, p in enumerate(prompts[:3])]
    ids = [sched.submit(np.array(p), GenerateConfig(len(p) + 6, strat, 5 + i)) for i, p in enumerate(prompts[:3])]
    done = {}
    for _ in range(40):
        sched.step()
        done.update(sched.take_finished())
    assert [done[i].tolist() for i in ids] == alone
    dec.close()


def test_verification_pass_returns_every_position():
    cfg = lc.config([lc.latent(window=9, mlp=lc.glu()), lc.latent(window=5, kv_from=0)])
    w = lc.weights(cfg, 17)
    toks = lc.tokens(cfg, 24, 1)
    want = oracle.forward(cfg, w, toks)
    dec = lc.make_decoder(ops(), cfg, w)
    dec.set_sequences(tables_of(dec, 1), [0])
    dec.prefill([toks[:10]])
    picked, logits = dec.verify([toks[10:]], want_logits=True)
    assert lc.error(logits[0], want[10:]) < F32_TOL
    assert picked[0].tolist() == want[10:].argmax(1).tolist()
    dec.rewind([12])                                       # no recurrent state: the sequence can be cut back
    assert lc.error(step_logits(dec, toks, 12, False), want[12:]) < F32_TOL
    dec.close()


def test_long_prompts_run_in_several_internal_passes():
    from fandhe_ai_amd.capi import lib
    cfg = lc.config(MECHANISMS["all"])
    w = lc.weights(cfg, 18)
    rows = [lc.tokens(cfg, n, 80 + n) for n in (150, 40, 90)]
    dec = lc.make_decoder(ops(), cfg, w)
    assert lib.fa_set_tuning(28, 64) == 0
    try:
        dec.set_sequences(tables_of(dec, 3), [0, 0, 0])
        want = [oracle.forward(cfg, w, r) for r in rows]
        got = dec.forward(rows, [[0, 63, 64, 149], [39], [1, 88]])
        ref = np.concatenate([want[0][[0, 63, 64, 149]], want[1][[39]], want[2][[1, 88]]])
        assert lc.error(got, ref) < F32_TOL
        dec.set_sequences(tables_of(dec, 3), [0, 0, 0])
        dec.prefill_padded(rows)
        assert lc.error(dec.logits(), np.array([x[-1] for x in want])) < F32_TOL
    finally:
        lib.fa_set_tuning(28, 0)
    dec.close()


def test_errors_are_reported_before_anything_runs():
    import fandhe_ai_amd as fa
    cfg = lc.config(MECHANISMS["all"][:3])
    w = lc.weights(cfg, 19)
    dec = fa.models.build_layered(ops(), cfg, "bfloat16", fa.models.Capacity(64, 2, 2))
    dec.set_sequences(tables_of(dec, 1), [0])
    with pytest.raises(fa.InvalidArgument, match="missing"):
        dec.step()
    with pytest.raises(fa.ShapeMismatch):
        dec.set_tensor("l0.norm1", np.zeros(3, np.float32))
    with pytest.raises(fa.InvalidArgument, match="no tensor"):
        dec.set_tensor("l9.norm1", np.zeros(3, np.float32))
    from fandhe_ai_amd.safetensors_io import MissingKeys, TypedTensor
    typed = {n: TypedTensor("F32", a.shape, a) for n, a in w.items()}
    with pytest.raises(fa.models.ConfigError, match="extra"):
        fa.models.install_weights(dec, dict(typed, extra=typed["embed"]))
    with pytest.raises(MissingKeys):
        fa.models.install_weights(dec, {n: t for n, t in typed.items() if n != "head"})
    fa.models.install_weights(dec, typed)
    with pytest.raises(fa.InvalidArgument, match="room"):
        dec.forward([[1] * 65])
    with pytest.raises(fa.InvalidArgument, match="vocabulary"):
        dec.forward([[10000]])
    with pytest.raises(fa.InvalidArgument, match="slot"):
        dec.set_state_slots([2])
    dec.forward([[1, 2, 3]])
    with pytest.raises(fa.Unsupported, match="recurrent"):
        dec.rewind([1])
    dec.close()
    bad = lc.config([lc.latent(), lc.latent(kv_from=0, kv_rank=8)])
    with pytest.raises(fa.InvalidArgument, match="kv_from"):
        fa.models.build_layered(ops(), bad, "bfloat16", fa.models.Capacity(64, 1))


def test_checkpoint_folder_trace_and_command_line(tmp_path, capsys):
    """config.json + model.safetensors through the registry, the trace replay and the command line's generation."""
    import io
    import json
    import types
    import fandhe_ai_amd as fa
    from fandhe_ai_amd import __main__ as cli
    from fandhe_ai_amd import trace
    cfg = lc.config(MECHANISMS["all"][:4])
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
