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


def test_grouped_attention_shares_heads_and_sees_the_past_only():
    rng = np.random.default_rng(3)
    q, k, v = rng.normal(size=(7, 4, 5)), rng.normal(size=(7, 2, 5)), rng.normal(size=(7, 2, 3))
    got = oracle.grouped_attention(q, k, v, 0.6)
    for t in range(7):
        for h in range(4):
            e = np.exp(0.6 * k[:t + 1, h // 2] @ q[t, h])
            assert np.allclose(got[t, h], e @ v[:t + 1, h // 2] / e.sum())


def test_projection_norm_runs_over_all_heads():
    rng = np.random.default_rng(4)
    mx = {"heads": 4, "kv_heads": 2, "dim": 3, "vdim": 2, "scale": 1.0}
    w = {"k": rng.normal(size=(6, 5)), "k.b": rng.normal(size=6), "k.norm": rng.normal(size=6), "v": rng.normal(size=(4, 5)), "v.b": rng.normal(size=4)}
    h = rng.normal(size=(3, 5))
    k, v = oracle.grouped_kv(h, w, "", mx, 1e-3)
    z = w["k"] @ h[1] + w["k.b"]
    assert np.allclose(k[1].ravel(), z / np.sqrt((z ** 2).mean() + 1e-3) * w["k.norm"])
    assert np.allclose(v[2].ravel(), w["v"] @ h[2] + w["v.b"])


def test_routing_takes_the_largest_and_weighs_them_among_themselves():
    z = np.array([[0.0, 3.0, 1.0, 2.0], [5.0, 5.0, -1.0, 4.0]])
    g = oracle.route(z, 2)
    assert np.allclose(g[0], [0, 1 / (1 + np.exp(-1)), 0, 1 / (1 + np.exp(1))])
    assert np.allclose(g[1], [0.5, 0.5, 0, 0])
    assert np.allclose(oracle.route(z, 4).sum(1), 1) and np.allclose(oracle.route(z, 1)[0], [0, 1, 0, 0])
    assert np.allclose(oracle.route_margin(z, 2) * z.std(axis=1), [1.0, 1.0]) and np.isinf(oracle.route_margin(z, 4)).all()
    w = {"router": np.array([[1.0], [0.0]]), "e0.up": np.array([[2.0]]), "e0.down": np.array([[3.0]]), "e1.up": np.array([[-1.0]]), "e1.down": np.array([[1.0]])}
    y = oracle.sparse_experts(np.array([[2.0], [-2.0]]), w, "", {"router": {"experts": 2, "top": 1}})
    assert np.allclose(y, [[48.0], [4.0]])


def test_additive_positions_closed_form():
    s = oracle.sinusoid([0, 7, 1000], 6)
    z = np.exp(1j * np.array([0, 7, 1000])[:, None] * 10000.0 ** (-2.0 * np.arange(3) / 6))
    assert np.allclose(s[:, 0::2], z.imag) and np.allclose(s[:, 1::2], z.real)
    assert oracle.sinusoid([5], 3).shape == (1, 3) and np.allclose(oracle.sinusoid([5], 3)[0, 2], np.sin(5 * 10000.0 ** (-2 / 3)))


def _change_mixers(cfg, key, value):
    for l in cfg["layers"]:
        l["mixer"][key] = value(l["mixer"][key])


ZOFERAX_MISTAKES = {
    "score scale": lambda c: _change_mixers(c, "scale", lambda s: s * 1.05),
    "norm eps": lambda c: c["norm"].update(eps=0.05),
    "embedding scale": lambda c: c["embedding"].update(scale=c["embedding"]["scale"] * 1.05),
    "one expert more": lambda c: [l["mlp"]["router"].update(top=l["mlp"]["router"]["top"] + 1) for l in c["layers"] if l["mlp"]],
    "cache of the wrong layer": lambda c: c["layers"][2]["mixer"].update(kv_from=1),
    "feed-forward left out": lambda c: c["layers"][0].update(mlp=None),
}


@pytest.mark.parametrize("name", sorted(ZOFERAX_MISTAKES))
def test_a_planted_mistake_in_a_zoferax_model_exceeds_the_gpu_tests_tolerance(name):
    cfg = lc.zoferax([lc.attention(mlp=lc.experts()), lc.attention(mlp=lc.experts(4, 1)), lc.attention(kv_from=0)])
    w = lc.weights(cfg, 5)
    toks = lc.tokens(cfg, 40, 5)
    good = oracle.forward(cfg, w, toks)
    wrong = copy.deepcopy(cfg)
    ZOFERAX_MISTAKES[name](wrong)
    assert lc.error(oracle.forward(wrong, w, toks), good) > 30 * 2e-4


@pytest.mark.parametrize("mistake", ["positions", "a key head each", "norm per head", "equal weights", "plain relu", "no bias"])
def test_another_reading_of_a_zoferax_mechanism_exceeds_the_gpu_tests_tolerance(mistake, monkeypatch):
    """The oracle with one mechanism computed otherwise."""
    cfg = lc.zoferax([lc.attention(mlp=lc.experts())])
    w = lc.weights(cfg, 5)
    toks = lc.tokens(cfg, 40, 5)
    good = oracle.forward(cfg, w, toks)
    if mistake == "positions":
        sinusoid = oracle.sinusoid
        monkeypatch.setattr(oracle, "sinusoid", lambda p, width: sinusoid(np.asarray(p) + 1, width))
    elif mistake == "a key head each":
        monkeypatch.setattr(oracle, "grouped_attention", lambda q, k, v, s: oracle.windowed_softmax_attention(
            q, np.tile(k, (1, q.shape[1] // k.shape[1], 1)), np.tile(v, (1, q.shape[1] // v.shape[1], 1)), s, len(q)))
    elif mistake == "norm per head":
        norm = oracle.rms_norm
        monkeypatch.setattr(oracle, "rms_norm", lambda x, g, eps: norm(x, g, eps) if x.shape[-1] == cfg["width"] else norm(x.reshape(len(x), -1, 20), 1.0, eps).reshape(x.shape) * g)
    elif mistake == "equal weights":
        route = oracle.route
        monkeypatch.setattr(oracle, "route", lambda z, top: (route(z, top) > 0) / top)
    elif mistake == "plain relu":
        monkeypatch.setattr(oracle, "squared_relu_expert", lambda h, v, p: np.maximum(h @ v[p + "up"].T, 0.0) @ v[p + "down"].T)
    else:
        w = dict(w, **{"l0.mix.k.b": np.zeros_like(w["l0.mix.k.b"])})
    assert lc.error(oracle.forward(cfg, w, toks), good) > 30 * 2e-4


# ---- Bubetar ------------------------------------------------------------------------------------------------------

def test_leading_rotation_of_either_layout_and_scaled_frequencies():
    rng = np.random.default_rng(6)
    x, pos = rng.normal(size=(4, 2, 10)), [0, 1, 7, 5000]
    for interleaved in (True, False):
        got = oracle.rotate_leading(x, pos, {"base": 50.0, "dims": 6}, interleaved)
        assert np.allclose(got[..., 6:], x[..., 6:]) and np.allclose(got[0], x[0])
        u, v = (np.arange(0, 6, 2), np.arange(1, 6, 2)) if interleaved else (np.arange(3), np.arange(3, 6))
        for i in range(3):
            a = np.array(pos) * 50.0 ** (-i / 3.0)
            c, s = np.cos(a)[:, None], np.sin(a)[:, None]
            assert np.allclose(got[..., u[i]], x[..., u[i]] * c - x[..., v[i]] * s) and np.allclose(got[..., v[i]], x[..., v[i]] * c + x[..., u[i]] * s)
    assert np.allclose(oracle.rotate_leading(x, pos, {"base": 50.0, "dims": 10}, False), oracle.rotate(x, pos, 50.0))
    turns = np.array([0.1, 1.0, 2.5, 4.0, 9.0])
    f = oracle.scaled_frequencies(turns * 2 * np.pi / 64, {"factor": 8.0, "low": 1.0, "high": 4.0, "original": 64}) * 64 / (2 * np.pi)
    assert np.allclose(f, [0.1 / 8, 1.0 / 8, 2.5 * (0.5 / 8 + 0.5), 4.0, 9.0])


def test_sink_takes_a_share_and_a_window_forgets():
    rng = np.random.default_rng(7)
    q, k, v = rng.normal(size=(6, 4, 5)), rng.normal(size=(6, 2, 5)), rng.normal(size=(6, 2, 3))
    assert np.allclose(oracle.sink_attention(q, k, v, 0.6), oracle.grouped_attention(q, k, v, 0.6))
    sink = rng.normal(size=4)
    got = oracle.sink_attention(q, k, v, 0.6, 3, sink)
    for t in range(6):
        lo = max(0, t - 2)
        for h in range(4):
            e = np.exp(0.6 * k[lo:t + 1, h // 2] @ q[t, h])
            assert np.allclose(got[t, h], e @ v[lo:t + 1, h // 2] / (e.sum() + np.exp(sink[h])))
    assert np.allclose(oracle.sink_attention(q, k, v, 0.6, 1), np.repeat(v, 2, axis=1))


def test_lightning_is_decayed_linear_attention():
    rng = np.random.default_rng(8)
    q, k, v, g = rng.normal(size=(7, 2, 4)), rng.normal(size=(7, 2, 4)), rng.normal(size=(7, 2, 3)), [0.6, 1.0]
    got = oracle.lightning_recurrence(q, k, v, g)
    for t in range(7):
        for h in range(2):
            assert np.allclose(got[t, h], sum(g[h] ** (t - s) * (q[t, h] @ k[s, h]) * v[s, h] for s in range(t + 1)))


def test_channel_decays_reduce_to_one_decay_and_act_on_key_channels():
    rng = np.random.default_rng(9)
    q, k, v = rng.normal(size=(7, 2, 4)), oracle.unit_vector(rng.normal(size=(7, 2, 4))), rng.normal(size=(7, 2, 3))
    beta, lg = rng.uniform(size=(7, 2)), -rng.uniform(size=(7, 2))
    assert np.allclose(oracle.channel_delta_recurrence(q, k, v, beta, np.repeat(lg[:, :, None], 4, axis=2)), oracle.delta_recurrence(q, k, v, beta, lg))
    # one write along two channels, then reads of each of them: every channel has faded by its own product
    k, q = np.zeros((4, 1, 2)), np.zeros((4, 1, 2))
    k[0, 0] = 0.6, 0.8
    q[:, 0, 0] = 1.0
    q[3, 0] = 0.0, 1.0
    lg = -rng.uniform(size=(4, 1, 2))
    got = oracle.channel_delta_recurrence(q, k, v[:4, :1], np.ones((4, 1)), lg)[:, 0]
    assert np.allclose(got[2], 0.6 * np.exp(lg[1:3, 0, 0].sum()) * v[0, 0]) and np.allclose(got[3], 0.8 * np.exp(lg[1:4, 0, 1].sum()) * v[0, 0])


def _mixers(c, kind):
    return [l["mixer"] for l in c["layers"] if l["type"] == kind]


BUBETAR_MISTAKES = {
    "scale of the left mixer": lambda c: [m.update(left_scale=m["left_scale"] * 1.05) for m in _mixers(c, "parallel")],
    "scale of the right mixer": lambda c: [m.update(right_scale=m["right_scale"] * 1.05) for m in _mixers(c, "parallel_2")],
    "scores, gated": lambda c: [m["left"].update(scale=m["left"]["scale"] * 1.05) for m in _mixers(c, "parallel")],
    "scores, key values": lambda c: [m["left"].update(scale=m["left"]["scale"] * 1.05) for m in _mixers(c, "parallel_2")],
    "scores, latent": lambda c: [m.update(scale=m["scale"] * 1.05) for m in _mixers(c, "latent_attention")],
    "rotation base": lambda c: [m["left"]["rot"].update(base=m["left"]["rot"]["base"] * 2) for m in _mixers(c, "parallel")],
    "rotated part": lambda c: [m["left"]["rot"].update(dims=m["left"]["rot"]["dims"] - 2) for m in _mixers(c, "parallel_2")],
    "no stretch": lambda c: [m["left"]["rot"].pop("scaling") for m in _mixers(c, "parallel_2")],
    "stretch of another context": lambda c: [m["left"]["rot"]["scaling"].update(original=60) for m in _mixers(c, "parallel_2")],
    "window one longer": lambda c: [m["left"]["mask"].update(size=m["left"]["mask"]["size"] + 1) for m in _mixers(c, "parallel_2")],
    "window one shorter": lambda c: [m["left"]["mask"].update(size=m["left"]["mask"]["size"] - 1) for m in _mixers(c, "parallel_2")],
    "decays of other heads": lambda c: [m["right"]["decay"].reverse() for m in _mixers(c, "parallel")],
    "logit scale": lambda c: c.update(logit_scale=c["logit_scale"] * 1.1),
    "soft cap": lambda c: c.update(logit_softcap=c["logit_softcap"] * 1.1),
    "norm eps": lambda c: c["norm"].update(eps=0.05),
    "feed-forward left out": lambda c: c["layers"][0].update(mlp=None),
}


def _bubetar():
    cfg = lc.bubetar([lc.parallel(mlp=lc.dense()), lc.parallel_2(), lc.open_latent()], softcap=4.0)
    return cfg, lc.weights(cfg, 5), lc.tokens(cfg, 40, 5)


@pytest.mark.parametrize("name", sorted(BUBETAR_MISTAKES))
def test_a_planted_mistake_in_a_bubetar_model_exceeds_the_gpu_tests_tolerance(name):
    cfg, w, toks = _bubetar()
    good = oracle.forward(cfg, w, toks)
    wrong = copy.deepcopy(cfg)
    BUBETAR_MISTAKES[name](wrong)
    assert lc.error(oracle.forward(wrong, w, toks), good) > 30 * 2e-4


@pytest.mark.parametrize("mistake", ["pairs of the other layout", "values behind the rotation", "a scaled sink", "no sink", "read before the write", "one decay for all channels",
                                     "norm per head", "the state forgotten", "relu"])
def test_another_reading_of_a_bubetar_mechanism_exceeds_the_gpu_tests_tolerance(mistake, monkeypatch):
    cfg, w, toks = _bubetar()
    good = oracle.forward(cfg, w, toks)
    rotate, attend, light, channel = oracle.rotate_leading, oracle.sink_attention, oracle.lightning_recurrence, oracle.channel_delta_recurrence
    if mistake == "pairs of the other layout":
        monkeypatch.setattr(oracle, "rotate_leading", lambda x, p, rot, interleaved: rotate(x, p, rot, not interleaved))
    elif mistake == "values behind the rotation":
        monkeypatch.setattr(oracle, "sink_attention", lambda q, k, v, s, window=None, sink=None: attend(q, k, v if sink is None else k, s, window, sink))
    elif mistake == "a scaled sink":
        monkeypatch.setattr(oracle, "sink_attention", lambda q, k, v, s, window=None, sink=None: attend(q, k, v, s, window, None if sink is None else sink * s))
    elif mistake == "no sink":
        monkeypatch.setattr(oracle, "sink_attention", lambda q, k, v, s, window=None, sink=None: attend(q, k, v, s, window))
    elif mistake == "read before the write":
        monkeypatch.setattr(oracle, "lightning_recurrence", lambda q, k, v, d: light(q, k, v, d) - (q * k).sum(-1, keepdims=True) * v)
    elif mistake == "one decay for all channels":
        monkeypatch.setattr(oracle, "channel_delta_recurrence", lambda q, k, v, b, g: channel(q, k, v, b, np.repeat(g.mean(2, keepdims=True), g.shape[2], axis=2)))
    elif mistake == "norm per head":
        norm = oracle.rms_norm
        n = cfg["layers"][0]["mixer"]["right"]
        monkeypatch.setattr(oracle, "rms_norm", lambda x, g, eps: norm(x, g, eps) if x.shape[-1] != n["heads"] * n["vdim"] else
                            norm(x.reshape(len(x), n["heads"], -1), 1.0, eps).reshape(x.shape) * g)
    elif mistake == "the state forgotten":
        monkeypatch.setattr(oracle, "lightning_recurrence", lambda q, k, v, d: np.concatenate([light(q[:20], k[:20], v[:20], d), light(q[20:], k[20:], v[20:], d)]))
    else:
        monkeypatch.setattr(oracle, "silu_glu", lambda h, v, p: (np.maximum(h @ v[p + "gate"].T, 0.0) * (h @ v[p + "up"].T)) @ v[p + "down"].T)
    assert lc.error(oracle.forward(cfg, w, toks), good) > 30 * 2e-4


# ---- Lugipel ---------------------------------------------------------------------------------------------------

def test_gated_recurrence_closed_forms():
    rng = np.random.default_rng(0)
    c = rng.normal(size=(9, 3))
    z = np.zeros((9, 3))
    z[2], z[5:, 1] = 1.0, 0.5
    S = oracle.gated_recurrence(z, c)
    assert (S[:2] == 0.0).all() and np.allclose(S[2:5], c[2]) and np.allclose(S[-1, 0], c[2, 0])       # written once, kept
    assert np.allclose(S[6, 1], 0.25 * c[2, 1] + 0.25 * c[5, 1] + 0.5 * c[6, 1])
    u = oracle.positive_candidate(np.array([-40.0, -1e-9, 0.0, 2.0]))
    assert np.allclose(u, [0.0, 0.5, 0.5, 2.5])


def test_sigmoid_attention_sums_what_it_sees():
    rng = np.random.default_rng(1)
    q, k, v = rng.normal(size=(12, 4, 5)), rng.normal(size=(12, 2, 5)), rng.normal(size=(12, 2, 3))
    slopes = oracle.distance_slopes(4)
    assert np.allclose(slopes, [0.25, 0.0625, 1 / 64.0, 1 / 256.0]) and np.allclose(oracle.distance_slopes(1), [2.0 ** -8])
    o = oracle.sigmoid_attention(q, k, v, 0.0, 4, 0.0 * slopes, np.full(4, 50.0))                       # every weight one
    assert np.allclose(o[9, 1], v[6:10, 0].sum(axis=0)) and np.allclose(o[2, 3], v[:3, 1].sum(axis=0))
    o = oracle.sigmoid_attention(q, k, v, 0.7, 1, slopes, np.zeros(4))
    assert np.allclose(o[5, 2], v[5, 1] / (1.0 + np.exp(-0.7 * q[5, 2] @ k[5, 1])))
    o = oracle.sigmoid_attention(q, 0.0 * k, v, 1.0, None, slopes, np.zeros(4))
    assert np.allclose(o[7, 0], sum(v[j, 0] / (1.0 + np.exp(0.25 * (7 - j))) for j in range(8)))


def test_query_temperature_steps_once_a_block_is_whole():
    t = oracle.query_temperature(range(20), 0.5, 8)
    assert (t[:7] == 1.0).all() and np.allclose(t[7:15], 1.0 + 0.5 * np.log(2.0)) and np.allclose(t[15:], 1.0 + 0.5 * np.log(3.0))


def test_xielu_closed_forms():
    p, q = np.log(np.expm1(0.8)), np.log(np.expm1(0.3))                # softplus gives 0.8 and 0.3
    z = np.array([-2.0, -1e-6, 0.0, 1.5])
    want = [0.8 * (np.exp(-2.0) + 1.0) - 1.0, -0.5e-6, 0.0, 0.8 * 2.25 + 0.75]
    assert np.allclose(oracle.xielu(z, p, q), want)


def test_experts_are_chosen_from_the_best_groups_by_corrected_scores():
    s = np.array([0.30, 0.05, 0.20, 0.10, 0.25, 0.10])
    none = np.zeros(6)
    assert sorted(oracle.grouped_choice(s, none, 3, 1, 1)[0]) == [0, 2, 4]
    assert sorted(oracle.grouped_choice(s, none, 3, 3, 2)[0]) == [0, 4, 5]          # the middle pair is left out
    assert sorted(oracle.grouped_choice(s, none - 1.0, 4, 3, 2)[0]) == [0, 1, 4, 5]  # and stays out where all are negative
    assert sorted(oracle.grouped_choice(s, np.array([-1.0, 0, 0, 1.0, 0, 0]), 2, 3, 1)[0]) == [2, 3]
    z = np.log(s)[None]
    g, _ = oracle.route_scored(z, np.array([-1.0, 0, 0, 1.0, 0, 0]), {"top": 2, "scale": 3.0, "groups": {"count": 3, "keep": 1}})
    assert np.allclose(g, [[0, 0, 2.0, 1.0, 0, 0]])                                 # weights know no correction
    rng = np.random.default_rng(2)
    h = rng.normal(size=(4, 5))
    w = {"m.router": np.zeros((3, 5)), "m.correction": np.array([0.0, 0.0, 1.0])}
    w.update({"m.e%d.%s" % (e, n): rng.normal(size=(5, 5)) for e in (0, 1) for n in ("gate", "up", "down")})
    y = oracle.scored_experts(h, w, "m.", {"router": {"experts": 2, "identity": 1, "top": 1, "scale": 0.5}})
    assert np.allclose(y, 0.5 * h)


def _lugipel():
    layers = [lc.sigmoid_attention(mlp=lc.dense(40)), lc.mingru(mlp=lc.scored()), lc.sigmoid_attention(heads=4, window=9, mlp=lc.scored(5, 3, (4, 2), 3)), lc.mingru(30)]
    cfg = lc.lugipel(layers)
    return cfg, lc.weights(cfg, 5), lc.tokens(cfg, 40, 5)


def _router(c, **change):
    for l in c["layers"]:
        if l["mlp"] and l["mlp"]["kind"] == "moe":
            l["mlp"]["router"].update(change)


LUGIPEL_MISTAKES = {
    "embedding scale": lambda c: c["embedding"].update(scale=c["embedding"]["scale"] * 1.05),
    "scores": lambda c: [m.update(scale=m["scale"] * 1.05) for m in _mixers(c, "attention")],
    "window one longer": lambda c: [m["mask"].update(size=m["mask"]["size"] + 1) for m in _mixers(c, "attention")],
    "window one shorter": lambda c: [m["mask"].update(size=m["mask"]["size"] - 1) for m in _mixers(c, "attention")],
    "temperature": lambda c: [m["q_temp"].update(coef=m["q_temp"]["coef"] * 1.1) for m in _mixers(c, "attention")],
    "temperature one position late": lambda c: [m["q_temp"].update(every=m["q_temp"]["every"] + 1) for m in _mixers(c, "attention")],
    "experts' scale": lambda c: _router(c, scale=1.7),
    "one expert fewer": lambda c: _router(c, top=2),
    "all groups kept": lambda c: [l["mlp"]["router"]["groups"].update(keep=l["mlp"]["router"]["groups"]["count"]) for l in c["layers"][1:3]],
    "no groups": lambda c: _router(c, groups=None),
    "norm eps": lambda c: c["norm"].update(eps=0.05),
    "feed-forward left out": lambda c: c["layers"][0].update(mlp=None),
}


@pytest.mark.parametrize("name", sorted(LUGIPEL_MISTAKES))
def test_a_planted_mistake_in_a_lugipel_model_exceeds_the_gpu_tests_tolerance(name):
    cfg, w, toks = _lugipel()
    good = oracle.forward(cfg, w, toks)
    wrong = copy.deepcopy(cfg)
    LUGIPEL_MISTAKES[name](wrong)
    assert lc.error(oracle.forward(wrong, w, toks), good) > 30 * 2e-4


def _without_groups_forgotten(s, correction, top, groups, keep):
    """Experts of the groups left out count as zero instead of minus infinity."""
    c = s + correction
    size = len(c) // groups
    best = np.argsort(-c.reshape(groups, size).max(axis=1), kind="stable")[:keep]
    c = np.where(np.repeat(np.isin(np.arange(groups), best), size), c, 0.0)
    return np.argsort(-c, kind="stable")[:top], np.inf


LUGIPEL_READINGS = {
    "softmax": ("sigmoid_attention", lambda f: lambda q, k, v, s, w, m, b: oracle.sink_attention(q, k, v, s, w)),
    "no distance": ("sigmoid_attention", lambda f: lambda q, k, v, s, w, m, b: f(q, k, v, s, w, 0 * m, b)),
    "slopes of other heads": ("sigmoid_attention", lambda f: lambda q, k, v, s, w, m, b: f(q, k, v, s, w, m[::-1], b)),
    "no bias per head": ("sigmoid_attention", lambda f: lambda q, k, v, s, w, m, b: f(q, k, v, s, w, m, 0 * b)),
    "a scaled bias": ("sigmoid_attention", lambda f: lambda q, k, v, s, w, m, b: f(q, k, v, s, w, m, s * b)),
    "weights that sum to one": ("sigmoid_attention", lambda f: lambda q, k, v, s, w, m, b: f(q, k, v, s, w, m, b) / f(q, k, np.ones_like(v), s, w, m, b)),
    "temperature from the position before": ("query_temperature", lambda f: lambda p, c, e: f([i - 1 for i in p], c, e)),
    "temperature that grows in between": ("query_temperature", lambda f: lambda p, c, e: np.array([1.0 + c * np.log((i + 1) / e + 1.0) for i in p])),
    "keep and write exchanged": ("gated_recurrence", lambda f: lambda z, c: f(1.0 - z, c)),
    "the state forgotten": ("gated_recurrence", lambda f: lambda z, c: np.concatenate([f(z[:20], c[:20]), f(z[20:], c[20:])])),
    "a bare candidate": ("positive_candidate", lambda f: lambda u: u),
    "a candidate without its half": ("positive_candidate", lambda f: lambda u: np.where(u >= 0.0, u, f(u))),
    "corrected weights": ("route_scored", lambda f: lambda z, c, r: f(z + c, 0 * c, r)),
    "groups left out count as zero": ("grouped_choice", lambda f: _without_groups_forgotten),
    "activation of p and q exchanged": ("xielu", lambda f: lambda z, p, q: f(z, q, p)),
    "activation without its half": ("xielu", lambda f: lambda z, p, q: f(z, p, q) - 0.5 * z),
    "norms that take the mean off": ("rms_norm", lambda f: oracle.layer_norm),
}


@pytest.mark.parametrize("mistake", sorted(LUGIPEL_READINGS))
def test_another_reading_of_a_lugipel_mechanism_exceeds_the_gpu_tests_tolerance(mistake, monkeypatch):
    cfg, w, toks = _lugipel()
    good = oracle.forward(cfg, w, toks)
    name, change = LUGIPEL_READINGS[mistake]
    monkeypatch.setattr(oracle, name, change(getattr(oracle, name)))
    assert lc.error(oracle.forward(cfg, w, toks), good) > 30 * 2e-4


@pytest.mark.parametrize("tensor", ["l0.mix.q.norm", "l0.mix.pb", "l0.mix.g", "l0.mlp.act", "l1.mix.z.b", "l1.mix.x.b", "l1.mlp.correction", "l3.mix.g", "final.norm"])
def test_every_small_tensor_of_a_lugipel_model_counts(tensor):
    cfg, w, toks = _lugipel()
    wrong = dict(w, **{tensor: np.roll(w[tensor], 1, axis=0)})
    assert lc.error(oracle.forward(cfg, wrong, toks), oracle.forward(cfg, w, toks)) > 30 * 2e-4


# ---- configuration ---------------------------------------------------------------------------------------------

def test_registry_picks_by_architecture_and_rejects_what_it_does_not_know(tmp_path):
    models = _fa().models
    assert {"Nugelix", "Zoferax", "Bubetar", "Lugipel", "LlamaForCausalLM"} <= set(models.ARCHITECTURES)
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


def test_zoferax_configuration_reads_every_size_and_names_what_is_missing():
    fa = _fa()
    models, capi = fa.models, fa.capi
    cfg = lc.zoferax([lc.attention(heads=12, kv_heads=4, dim=10, vdim=6, scale=0.25, mlp=lc.experts(7, 3, 44)), lc.attention(kv_from=0)], scale=2.5)
    a = models.zoferax(cfg)
    assert (a["d_model"], a["vocab"], a["norm"], a["embed_scale"], a["position_base"], a["norm_eps"]) == (76, 131, capi.NORM_OUTPUT, 2.5, 10000.0, 1e-5)
    l, m = a["layers"]
    assert (l["mixer"], l["heads"], l["kv_heads"], l["dim"], l["vdim"], l["scale"], l["kv_from"]) == (capi.MIXER_ATTENTION, 12, 4, 10, 6, 0.25, -1)
    assert (l["d_ffn"], l["experts"], l["top"]) == (44, 7, 3) and m["kv_from"] == 0 and "d_ffn" not in m
    for path in (("mixer", "kv_heads"), ("mixer", "scale"), ("type",), ("mlp", "kind"), ("mlp", "router", "top"), ("mlp", "expert", "ff")):
        bad = copy.deepcopy(cfg)
        at = bad["layers"][0]
        for key in path[:-1]:
            at = at[key]
        del at[path[-1]]
        with pytest.raises(models.ConfigError, match=path[-1]):
            models.zoferax(bad)
    for change in ({"type": "delta"}, {"mlp": {"kind": "dense", "ff": 3}}):
        bad = copy.deepcopy(cfg)
        bad["layers"][1].update(change)
        with pytest.raises(models.ConfigError, match="unknown"):
            models.zoferax(bad)


def test_bubetar_configuration_reads_every_size_and_names_what_is_missing():
    fa = _fa()
    models, capi = fa.models, fa.capi
    cfg = lc.bubetar([lc.parallel(mlp=lc.dense(44)), lc.parallel_2(), lc.open_latent()], scale=0.3, ranks=(7, 11))
    shapes = lc.shapes(cfg)
    a = models.bubetar(cfg, shapes)
    assert (a["d_model"], a["vocab"], a["norm"], a["logit_scale"], a["logit_softcap"], a["norm_eps"]) == (76, 131, capi.NORM_BOTH, 0.3, 12.0, 1e-5)
    p, q, l = a["layers"]
    assert (p["mixer"], p["heads"], p["kv_heads"], p["dim"], p["vdim"], p["rot_dim"], p["rot_base"], p["rot_interleaved"]) == (capi.MIXER_ATTENTION, 6, 2, 20, 12, 12, 3000.0, 1)
    assert p["attention"] == capi.ATTENTION_HEAD_NORM | capi.ATTENTION_GATE and p.get("window", 0) == 0 and "rot_factor" not in p
    assert (p["left_scale"], p["right_scale"], p["d_ffn"], p["glu"]) == (0.7, 1.3, 44, capi.GLU_SILU)
    r = p["right"]
    assert (r["mixer"], r["heads"], r["dim"], r["vdim"], len(r["decay"])) == (capi.MIXER_LIGHTNING, 3, 20, 28, 3)
    assert q["attention"] == capi.ATTENTION_HEAD_UNIT | capi.ATTENTION_KEY_VALUES | capi.ATTENTION_SINK and (q["window"], q["rot_interleaved"]) == (11, 0)
    assert (q["rot_factor"], q["rot_low"], q["rot_high"], q["rot_original"]) == (6.0, 1.0, 3.0, 90) and q.get("d_ffn", 0) == 0
    r = q["right"]
    assert (r["mixer"], r["kv_heads"], r["conv"], r["decay_rank"], r["gate_rank"]) == (capi.MIXER_DELTA, 2, 4, 7, 11)
    assert (l["mixer"], l["ungated"], l["q_rank"], l["kv_rank"], l["rot_dim"], l.get("window", 0), l["rot_interleaved"]) == (capi.MIXER_LATENT_ATTENTION, 1, 36, 44, 12, 0, 1)
    for layer, path in ((0, ("mixer", "left", "scale")), (0, ("mixer", "right", "decay")), (0, ("mixer", "left_scale")), (1, ("mixer", "right", "conv")),
                        (1, ("mixer", "left", "rot", "scaling", "low")), (2, ("mixer", "q_rank")), (2, ("mixer", "rot", "dims")), (0, ("mlp", "ff")), (1, ("type",))):
        bad = copy.deepcopy(cfg)
        at = bad["layers"][layer]
        for key in path[:-1]:
            at = at[key]
        del at[path[-1]]
        with pytest.raises(models.ConfigError, match=path[-1]):
            models.bubetar(bad, shapes)
    with pytest.raises(models.ConfigError, match="a1"):
        models.bubetar(cfg, {})
    for change, word in (({"type": "other"}, "unknown type"), ({"mlp": {"kind": "moe"}}, "unknown feed-forward")):
        bad = copy.deepcopy(cfg)
        bad["layers"][2].update(change)
        with pytest.raises(models.ConfigError, match=word):
            models.bubetar(bad, shapes)
    bad = copy.deepcopy(cfg)
    bad["layers"][0]["mixer"]["right"]["decay"].pop()
    with pytest.raises(models.ConfigError, match="decay"):
        models.bubetar(bad, shapes)


def test_lugipel_configuration_reads_every_size_and_names_what_is_missing():
    fa = _fa()
    models, capi = fa.models, fa.capi
    cfg = lc.lugipel([lc.sigmoid_attention(heads=12, kv_heads=4, dim=10, vdim=6, window=21, scale=0.25, coef=0.3, every=5, mlp=lc.dense(44)),
                      lc.mingru(37, mlp=lc.scored(7, 5, (4, 3), 6, 18, 0.7)), lc.mingru(8, mlp=lc.scored(4, 0, None, 2, 9, 1.0)), lc.sigmoid_attention()], scale=2.5)
    a = models.lugipel(cfg)
    assert (a["d_model"], a["vocab"], a["norm"], a["embed_scale"], a["position_base"], a["norm_eps"]) == (76, 131, capi.NORM_INPUT_RMS, 2.5, 10000.0, 1e-5)
    p, q, r, s = a["layers"]
    assert (p["mixer"], p["heads"], p["kv_heads"], p["dim"], p["vdim"], p["scale"], p["window"]) == (capi.MIXER_ATTENTION, 12, 4, 10, 6, 0.25, 21)
    assert p["attention"] == capi.ATTENTION_HEAD_NORM | capi.ATTENTION_SIGMOID | capi.ATTENTION_HEAD_GATE and p.get("rot_dim", 0) == 0
    assert (p["distance"], p["q_temp"], p["q_temp_every"], p["d_ffn"], p["glu"]) == (8.0, 0.3, 5, 44, capi.FFN_XIELU)
    assert (q["mixer"], q["heads"], q["vdim"]) == (capi.MIXER_MINGRU, 1, 37)
    assert (q["experts"], q["identity"], q["top"], q["groups"], q["groups_kept"], q["d_ffn"], q["route_scale"]) == (12, 5, 6, 4, 3, 18, 0.7)
    assert (q["route"], q["glu"]) == (capi.ROUTE_SCORED, capi.GLU_SILU)
    assert (r["experts"], r["identity"], r["top"], r.get("groups", 0)) == (4, 0, 2, 0) and "d_ffn" not in s
    for layer, path in ((0, ("mixer", "kv_heads")), (0, ("mixer", "q_temp", "every")), (0, ("mixer", "mask", "size")), (0, ("mlp", "ff")), (1, ("mixer", "width")),
                        (1, ("mlp", "router", "scale")), (1, ("mlp", "router", "groups", "keep")), (1, ("mlp", "expert", "ff")), (2, ("type",)), (0, ("mlp", "kind"))):
        bad = copy.deepcopy(cfg)
        at = bad["layers"][layer]
        for key in path[:-1]:
            at = at[key]
        del at[path[-1]]
        with pytest.raises(models.ConfigError, match=path[-1]):
            models.lugipel(bad)
    for change in ({"type": "delta"}, {"mlp": {"kind": "glu", "ff": 3}}):
        bad = copy.deepcopy(cfg)
        bad["layers"][1].update(change)
        with pytest.raises(models.ConfigError, match="unknown"):
            models.lugipel(bad)
    bad = copy.deepcopy(cfg)
    bad["layers"][0]["mixer"]["q_temp"]["every"] = 2.5
    with pytest.raises(models.ConfigError, match="every"):
        models.lugipel(bad)
    bare = models.lugipel_layers(lc.lugipel([lc.sigmoid_attention(window=None, every=None)]))[0]
    assert bare.get("window", 0) == 0 and bare.get("q_temp", 0.0) == 0.0


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
