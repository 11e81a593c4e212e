"""CPU side of the layered decoders: the oracle's mechanisms against closed forms, that the comparisons of the GPU tests
would see a planted mistake, the registry's configuration checks, and the batchers' bookkeeping on a fake decoder."""
import copy
import json

import numpy as np
import pytest

import layered_common as lc
from layered_common import oracle


def _fa():
    import fandhe_ai_amd as fa
    return fa


# ---- the oracle's mechanisms ------------------------------------------------------------------------------------

def test_delta_recurrence_closed_forms():
    rng = np.random.default_rng(0)
    T, dk, dv = 6, 5, 3
    v = rng.normal(size=(T, 1, dv))
    # orthonormal keys, full writes, no decay: reading with key j returns value j as soon as it was written
    k = np.eye(dk + 1)[:T, None, :]
    out = oracle.delta_recurrence(k, k, v, np.ones((T, 1)), np.zeros((T, 1)))
    assert np.allclose(out, v)
    # the same key again replaces the value
    k = np.repeat(np.eye(dk)[:1, None, :], T, axis=0)
    assert np.allclose(oracle.delta_recurrence(k, k, v, np.ones((T, 1)), np.zeros((T, 1))), v)
    # decay: a value written once and read n tokens later has shrunk by the product of the decays
    lg = rng.uniform(-1, 0, (T, 1))
    k = np.eye(dk + 1)[:T, None, :]
    q = np.repeat(np.eye(dk + 1)[:1, None, :], T, axis=0)
    out = oracle.delta_recurrence(q, k, v, np.ones((T, 1)), lg)
    assert np.allclose(out[:, 0], v[0, 0] * np.exp(np.cumsum(lg[:, 0]) - lg[0, 0])[:, None])


def test_convolution_rotation_and_norms_closed_forms():
    rng = np.random.default_rng(1)
    x, taps = rng.normal(size=(7, 3)), rng.normal(size=(3, 4))
    y = oracle.causal_conv(x, taps)
    for t in range(7):
        want = sum(taps[:, 3 - b] * x[t - b] for b in range(4) if t - b >= 0)
        assert np.allclose(y[t], want)
    r = rng.normal(size=(5, 2, 8))
    pos = np.array([0, 1, 5, 900, 70000])
    rot = oracle.rotate(r, pos, 500.0)
    assert np.allclose(rot[0], r[0])
    assert np.allclose((rot ** 2).sum(-1), (r ** 2).sum(-1))
    z = (r[..., :4] + 1j * r[..., 4:]) * np.exp(1j * pos[:, None, None] * 500.0 ** (-np.arange(4) / 4.0))
    assert np.allclose(rot, np.concatenate([z.real, z.imag], axis=-1))
    n = oracle.layer_norm(x, np.ones(3), 0.0)
    assert np.allclose(n.mean(-1), 0) and np.allclose((n ** 2).mean(-1), 1)
    assert np.allclose(oracle.rms_norm(np.array([[1.0, 2.0, 3.0, 4.0]]), 1.0, 0.0), np.arange(1, 5) / np.sqrt(7.5))


def test_window_of_one_returns_the_tokens_own_value():
    rng = np.random.default_rng(2)
    q, k, v = rng.normal(size=(6, 2, 4)), rng.normal(size=(6, 2, 4)), rng.normal(size=(6, 2, 3))
    assert np.allclose(oracle.windowed_softmax_attention(q, k, v, 1.0, 1), v)
    whole = oracle.windowed_softmax_attention(q, k, v, 0.7, 100)
    s = np.exp(0.7 * np.einsum("ihd,jhd->hij", q, k)) * np.tril(np.ones((6, 6)))
    assert np.allclose(whole, np.einsum("hij,jhd->ihd", s / s.sum(-1, keepdims=True), v))


def test_clamped_glu_and_softcap():
    w = {"gate": np.array([[1.0]]), "up": np.array([[1.0]]), "down": np.array([[1.0]])}
    for x in (-5.0, 0.3, 5.0):
        g, u = min(x, 2.0), max(-2.0, min(x, 2.0))
        assert np.allclose(oracle.clamped_glu(np.array([[x]]), w, "", 2.0), g / (1 + np.exp(-1.702 * g)) * (u + 1))
    assert abs(oracle.softcap(1e9, 7.0) - 7.0) < 1e-9 and abs(oracle.softcap(1e-3, 7.0) - 1e-3) < 1e-9


MISTAKES = {
    "window one longer": lambda c: [l["mixer"]["mask"].update(size=l["mixer"]["mask"]["size"] + 1) for l in c["layers"] if "mask" in l["mixer"]],
    "window one shorter": lambda c: [l["mixer"]["mask"].update(size=l["mixer"]["mask"]["size"] - 1) for l in c["layers"] if "mask" in l["mixer"]],
    "score scale": lambda c: [l["mixer"].update(scale=l["mixer"]["scale"] * 1.05) for l in c["layers"] if "mask" in l["mixer"]],
    "rotation base": lambda c: [l["mixer"]["rot"].update(base=l["mixer"]["rot"]["base"] * 2) for l in c["layers"] if "mask" in l["mixer"]],
    "clamp limit": lambda c: [l["mlp"].update(limit=l["mlp"]["limit"] * 1.1) for l in c["layers"] if l["mlp"]],
    "soft cap": lambda c: c.update(logit_softcap=c["logit_softcap"] * 1.1),
    "cache of the wrong layer": lambda c: c["layers"][3]["mixer"].update(kv_from=2),
    "norm eps": lambda c: c["norm"].update(eps=0.05),
}


@pytest.mark.parametrize("name", sorted(MISTAKES))
def test_a_planted_mistake_exceeds_the_gpu_tests_tolerance(name):
    """The oracle with one constant wrong differs from the right one by far more than the GPU tests (f32) allow."""
    cfg = lc.config([lc.latent(window=9, mlp=lc.glu()), lc.delta(), lc.latent(window=6), lc.latent(window=7, kv_from=0)], softcap=4.0)
    w = lc.weights(cfg, 5)
    toks = lc.tokens(cfg, 40, 5)
    good = oracle.forward(cfg, w, toks)
    wrong = copy.deepcopy(cfg)
    MISTAKES[name](wrong)
    assert lc.error(oracle.forward(wrong, w, toks), good) > 30 * 2e-4


# ---- configuration ---------------------------------------------------------------------------------------------

def test_registry_picks_by_architecture_and_rejects_what_it_does_not_know(tmp_path):
    models = _fa().models
    assert {"Nugelix", "LlamaForCausalLM"} <= set(models.ARCHITECTURES)
    (tmp_path / "config.json").write_text(json.dumps({"architecture": "Nonesuch"}))
    with pytest.raises(models.ConfigError, match="unknown architecture"):
        models.load_model(None, str(tmp_path))
    with pytest.raises(models.ConfigError, match="dtype"):
        models.load_model(None, str(tmp_path), "float16")
    with pytest.raises(models.ConfigError):
        models.read_config(str(tmp_path / "missing"))


def test_layer_list_reads_every_size_and_names_what_is_missing():
    fa = _fa()
    models, capi = fa.models, fa.capi
    cfg = lc.config([lc.latent(window=5, base=300.0, mlp=lc.glu(40, 0.7)), lc.delta(conv=2), lc.latent(kv_from=0, scale=0.4)])
    a, b, c = models.nugelix_layers(cfg)
    assert (a["mixer"], a["window"], a["rot_base"], a["d_ffn"], a["ffn_limit"], a["kv_from"]) == (capi.MIXER_LATENT_ATTENTION, 5, 300.0, 40, 0.7, -1)
    assert (b["mixer"], b["kv_heads"], b["conv"], b.get("d_ffn", 0)) == (capi.MIXER_DELTA, 2, 2, 0)
    assert (c["kv_from"], c["scale"]) == (0, 0.4)
    for path in (("mixer", "kv_rank"), ("mixer", "mask"), ("type",)):
        bad = copy.deepcopy(cfg)
        at = bad["layers"][0]
        for key in path[:-1]:
            at = at[key]
        del at[path[-1]]
        with pytest.raises(models.ConfigError, match=path[-1]):
            models.nugelix_layers(bad)
    bad = copy.deepcopy(cfg)
    bad["layers"][0]["mixer"]["rot"]["dims"] = 6
    with pytest.raises(models.ConfigError, match="rot_dim"):
        models.nugelix_layers(bad)
    bad = copy.deepcopy(cfg)
    bad["layers"][1]["type"] = "other"
    with pytest.raises(models.ConfigError, match="unknown type"):
        models.nugelix_layers(bad)


# ---- batching on a fake decoder ---------------------------------------------------------------------------------

class FakeDecoder:
    """Next token = (last token + 1) mod vocab; a slot's history must be its sequence's own."""
    takes_portions = True

    class cfg:
        vocab, block_size, max_blocks_per_seq, num_blocks, max_batch, n_layers, d_model = 50, 4, 6, 6, 3, 1, 1

    def __init__(self, state_slots=3):
        self.state_slots, self.calls, self.history = state_slots, [], {}

    def set_sequences(self, tables, lens):
        self.tables, self.lens, self.batch = np.array(tables), list(lens), len(lens)

    def set_state_slots(self, slots):
        assert len(set(slots)) == len(slots) == self.batch and max(slots) < self.state_slots
        self.slots = list(slots)

    def forward(self, portions, want):
        out = []
        used = []
        for b, p in enumerate(portions):
            if self.lens[b] == 0:
                self.history[self.slots[b]] = []
            h = self.history[self.slots[b]]
            assert len(h) == self.lens[b]
            h.extend(p)
            used.extend(self.tables[b, :-(-len(h) // self.cfg.block_size)])
            out += [np.eye(self.cfg.vocab)[(p[k] + 1) % self.cfg.vocab] for k in want[b]]
        assert len(set(used)) == len(used) and all(u < self.cfg.num_blocks for u in used)
        return np.array(out, dtype=np.float32).reshape(len(out), self.cfg.vocab)


def test_portion_batcher_takes_pages_as_requests_grow_and_reuses_them():
    sched = _fa().scheduler
    dec = FakeDecoder()
    b = sched.PortionBatcher(dec)
    assert b.feed([("a", [1, 2, 3], [2]), ("b", [7], [])]).argmax(1).tolist() == [4]
    assert b.free_pages() == 4 and b.live() == ["a", "b"]
    b.feed([("a", [4, 5], [0, 1])])
    assert b.free_pages() == 3
    slot_a = b._live["a"][2]
    b.release("a")
    assert b.free_pages() == 5
    b.feed([("b", [8] * 4, [3]), ("c", [9], [0])])            # b goes on after a step without it
    assert b._live["c"][2] == slot_a and b.free_pages() == 3
    with pytest.raises(sched.InvalidArgument, match="fit"):
        b.feed([("c", [1] * 20, [])])
    assert b.free_pages() == 3 and b._live["c"][0] == 1       # unchanged
    for bad in ([("c", [], [])], [("c", [50], [])], [("c", [1], [1])], [("c", [1, 2], [1, 0])], [("c", [1], []), ("c", [1], [])], []):
        with pytest.raises(sched.InvalidArgument):
            b.feed(bad)
    with pytest.raises(sched.InvalidArgument):
        b.release("zzz")


def test_portion_batcher_runs_out_of_state_slots():
    sched = _fa().scheduler
    b = sched.PortionBatcher(FakeDecoder(state_slots=1))
    b.feed([("a", [1], [])])
    with pytest.raises(sched.InvalidArgument, match="fit"):
        b.feed([("b", [1], [])])
    b.release("a")
    b.feed([("b", [1], [])])


def test_speculative_decoding_refuses_recurrent_states():
    sched = _fa().scheduler
    cfg = sched.GenerateConfig(8, sched.SamplingStrategy.Greedy())
    with pytest.raises(sched.InvalidArgument, match="recurrent"):
        sched.generate_speculative(FakeDecoder(), FakeDecoder(), [1, 2], cfg, 2)
