"""Small random layered models for the tests: configuration, bf16-representable weights, the oracle's logits, and a
decoder holding the same model."""
import os
import sys

import numpy as np

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
sys.path.insert(0, os.path.join(ROOT, "oracle"))
import layered as oracle  # noqa: E402


def delta(heads=4, kv_heads=2, dim=24, vdim=20, conv=4, mlp=None):
    return {"type": "delta", "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv}, "mlp": mlp}


def latent(heads=3, dim=20, rot=12, vdim=28, q_rank=36, kv_rank=44, window=13, scale=None, base=10000.0, kv_from=None, mlp=None):
    mx = {"heads": heads, "dim": dim, "rot_dim": rot, "vdim": vdim, "q_rank": q_rank, "kv_rank": kv_rank, "mask": {"size": window},
          "rot": {"base": base, "dims": rot}, "scale": (dim + rot) ** -0.5 if scale is None else scale}
    if kv_from is not None:
        mx["kv_from"] = kv_from
    return {"type": "latent_attention", "mixer": mx, "mlp": mlp}


def glu(ff=52, limit=1.5):
    return {"kind": "dense", "ff": ff, "limit": limit}


def config(layers, width=76, vocab=131, eps=1e-5, softcap=12.0):
    return {"architecture": "Nugelix", "width": width, "vocab": vocab, "layers": layers, "norm": {"eps": eps}, "logit_softcap": softcap}


def attention(heads=6, kv_heads=2, dim=20, vdim=12, scale=None, kv_from=None, mlp=None):
    mx = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": 2.0 * dim ** -0.5 if scale is None else scale}
    if kv_from is not None:
        mx["kv_from"] = kv_from
    return {"type": "attention", "mixer": mx, "mlp": mlp}


def experts(n=5, top=2, ff=28):
    return {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": n, "top": top}}


def zoferax(layers, width=76, vocab=131, eps=1e-5, scale=1.7):
    return {"architecture": "Zoferax", "width": width, "vocab": vocab, "layers": layers, "norm": {"eps": eps}, "embedding": {"scale": scale}}


def rotation(dims, base=10000.0, scaling=None):
    rot = {"base": base, "dims": dims}
    if scaling:
        rot["scaling"] = dict(zip(("factor", "low", "high", "original"), scaling))
    return rot


def beside(left, right, kind, scales, mlp):
    return {"type": kind, "mixer": {"left": left, "right": right, "left_scale": scales[0], "right_scale": scales[1]}, "mlp": mlp}


def gated_left(heads=6, kv_heads=2, dim=20, vdim=12, rot=12, scale=None, base=3000.0):
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "rot": rotation(rot, base), "scale": 1.4 * dim ** -0.5 if scale is None else scale}


def lightning_right(heads=3, dim=20, vdim=28, decay=None):
    return {"heads": heads, "dim": dim, "vdim": vdim, "decay": [1.0 - 0.7 ** (2 * h + 1) for h in range(heads)] if decay is None else decay}


def key_value_left(heads=6, kv_heads=3, dim=20, rot=16, window=11, scale=None, base=5000.0, scaling=(6.0, 1.0, 3.0, 90)):
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "rot": rotation(rot, base, scaling), "mask": {"size": window},
            "scale": 1.3 * dim ** -0.5 if scale is None else scale}


def channel_right(heads=4, kv_heads=2, dim=20, vdim=12, conv=4):
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv}


def parallel(left=None, right=None, scales=(0.7, 1.3), mlp=None):
    return beside(left or gated_left(), right or lightning_right(), "parallel", scales, mlp)


def parallel_2(left=None, right=None, scales=(1.4, 0.6), mlp=None):
    return beside(left or key_value_left(), right or channel_right(), "parallel_2", scales, mlp)


def open_latent(heads=3, dim=20, rot=12, vdim=28, q_rank=36, kv_rank=44, scale=None, base=10000.0, mlp=None):
    l = latent(heads, dim, rot, vdim, q_rank, kv_rank, 1, scale, base, None, mlp)
    del l["mixer"]["mask"]
    return l


def dense(ff=52):
    return {"kind": "dense", "ff": ff}


def bubetar(layers, width=76, vocab=131, eps=1e-5, softcap=12.0, scale=0.8, ranks=(10, 14)):
    """ranks: of the low-rank decays and gates, which only the weights' shapes tell."""
    return {"architecture": "Bubetar", "width": width, "vocab": vocab, "layers": layers, "norm": {"eps": eps}, "logit_scale": scale, "logit_softcap": softcap,
            "_ranks": ranks}


def sigmoid_attention(heads=6, kv_heads=2, dim=20, vdim=12, window=13, scale=None, coef=0.6, every=8, mlp=None):
    mx = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": 1.5 * dim ** -0.5 if scale is None else scale}
    if window:
        mx["mask"] = {"size": window}
    if every:
        mx["q_temp"] = {"coef": coef, "every": every}
    return {"type": "attention", "mixer": mx, "mlp": mlp}


def mingru(width=52, mlp=None):
    return {"type": "mingru", "mixer": {"width": width}, "mlp": mlp}


def scored(n=6, identity=3, groups=(3, 2), top=3, ff=28, scale=1.6):
    """groups: count and those kept; None for none."""
    router = {"experts": n, "top": top, "scale": scale}
    if identity:
        router["identity"] = identity
    if groups:
        router["groups"] = {"count": groups[0], "keep": groups[1]}
    return {"kind": "moe", "expert": {"ff": ff}, "router": router}


def lugipel(layers, width=76, vocab=131, eps=1e-5, scale=1.7):
    return {"architecture": "Lugipel", "width": width, "vocab": vocab, "layers": layers, "norm": {"eps": eps}, "embedding": {"scale": scale}}


def bf16_round(a):
    u = np.ascontiguousarray(a, dtype=np.float32).view(np.uint32)
    return ((u + 0x7FFF + ((u >> 16) & 1)) & 0xFFFF0000).astype(np.uint32).view(np.float32)


def zoferax_shapes(cfg):
    D = cfg["width"]
    out = {"embed": (cfg["vocab"], D), "head": (cfg["vocab"], D), "final.norm": (D,)}
    for i, l in enumerate(cfg["layers"]):
        p, mx = "l%d." % i, l["mixer"]
        q, k, v = (mx[h] * mx[d] for h, d in (("heads", "dim"), ("kv_heads", "dim"), ("kv_heads", "vdim")))
        out.update({p + "norm1": (D,), p + "mix.q": (q, D), p + "mix.q.b": (q,), p + "mix.q.norm": (q,), p + "mix.o": (D, mx["heads"] * mx["vdim"])})
        if "kv_from" not in mx:
            out.update({p + "mix.k": (k, D), p + "mix.k.b": (k,), p + "mix.k.norm": (k,), p + "mix.v": (v, D), p + "mix.v.b": (v,)})
        if l["mlp"]:
            n, ff = l["mlp"]["router"]["experts"], l["mlp"]["expert"]["ff"]
            out.update({p + "norm2": (D,), p + "mlp.router": (n, D)})
            for e in range(n):
                out.update({p + "mlp.e%d.up" % e: (ff, D), p + "mlp.e%d.down" % e: (D, ff)})
    return out


def bubetar_shapes(cfg):
    D = cfg["width"]
    out = {"embed": (cfg["vocab"], D), "head": (cfg["vocab"], D), "final.norm": (D,)}
    for i, l in enumerate(cfg["layers"]):
        p, mx = "l%d." % i, l["mixer"]
        out.update({p + "norm1": (D,), p + "norm1b": (D,)})
        if l["type"] == "latent_attention":
            m, H, r, k, d = p + "mix.", mx["heads"], mx["q_rank"], mx["kv_rank"], mx["dim"]
            out.update({m + "dq": (r, D), m + "dq.norm": (r,), m + "uq": (H * (d + mx["rot_dim"]), r), m + "dkv": (k + mx["rot_dim"], D),
                        m + "dkv.norm": (k,), m + "uk": (H * d, k), m + "uv": (H * mx["vdim"], k), m + "o": (D, H * mx["vdim"])})
        else:
            a, b, m, n = mx["left"], mx["right"], p + "mix.left.", p + "mix.right."
            H, G, d, wide = a["heads"], a["kv_heads"], a["dim"], b["heads"] * b["vdim"]
            out.update({m + "q": (H * d, D), m + "k": (G * d, D), m + "o": (D, H * a["vdim"]), n + "v": (wide, D), n + "o": (D, wide)})
            if l["type"] == "parallel":
                out.update({m + "v": (G * a["vdim"], D), m + "q.norm": (d,), m + "k.norm": (d,), m + "g": (H * a["vdim"], D), n + "q": (b["heads"] * b["dim"], D),
                            n + "k": (b["heads"] * b["dim"], D), n + "g": (wide, D), n + "norm": (wide,)})
            else:
                (ra, rg), nq, nd = cfg["_ranks"], b["kv_heads"] * b["dim"], b["heads"] * b["dim"]
                out.update({m + "sink": (H,), n + "q": (nq, D), n + "k": (nq, D), n + "q.conv": (nq, b["conv"]), n + "k.conv": (nq, b["conv"]),
                            n + "v.conv": (wide, b["conv"]), n + "b": (b["heads"], D), n + "A_log": (b["heads"],), n + "dt_bias": (nd,), n + "norm": (b["vdim"],),
                            n + "a1": (ra, D), n + "a2": (nd, ra), n + "g1": (rg, D), n + "g2": (wide, rg)})
        if l["mlp"]:
            f, ff = p + "mlp.", l["mlp"]["ff"]
            out.update({p + "norm2": (D,), p + "norm2b": (D,), f + "gate": (ff, D), f + "up": (ff, D), f + "down": (D, ff)})
    return out


def lugipel_shapes(cfg):
    D = cfg["width"]
    out = {"embed": (cfg["vocab"], D), "head": (cfg["vocab"], D), "final.norm": (D,)}
    for i, l in enumerate(cfg["layers"]):
        p, m, f, mx = "l%d." % i, "l%d.mix." % i, "l%d.mlp." % i, l["mixer"]
        out[p + "norm1"] = (D,)
        if l["type"] == "mingru":
            wide = mx["width"]
            out.update({m + "z": (wide, D), m + "z.b": (wide,), m + "x": (wide, D), m + "x.b": (wide,), m + "g": (wide, D), m + "o": (D, wide)})
        else:
            H, G, d, v = mx["heads"], mx["kv_heads"], mx["dim"], mx["vdim"]
            out.update({m + "q": (H * d, D), m + "k": (G * d, D), m + "v": (G * v, D), m + "q.norm": (d,), m + "k.norm": (d,), m + "pb": (H,), m + "g": (H, D),
                        m + "o": (D, H * v)})
        if not l["mlp"]:
            continue
        out[p + "norm2"] = (D,)
        if l["mlp"]["kind"] == "dense":
            out.update({f + "up": (l["mlp"]["ff"], D), f + "down": (D, l["mlp"]["ff"]), f + "act": (2,)})
        else:
            r, ff = l["mlp"]["router"], l["mlp"]["expert"]["ff"]
            n = r["experts"] + r.get("identity", 0)
            out.update({f + "router": (n, D), f + "correction": (n,)})
            for e in range(r["experts"]):
                out.update({f + "e%d.gate" % e: (ff, D), f + "e%d.up" % e: (ff, D), f + "e%d.down" % e: (D, ff)})
    return out


def shapes(cfg):
    if cfg["architecture"] == "Lugipel":
        return lugipel_shapes(cfg)
    if cfg["architecture"] == "Bubetar":
        return bubetar_shapes(cfg)
    if cfg["architecture"] == "Zoferax":
        return zoferax_shapes(cfg)
    D = cfg["width"]
    out = {"embed": (cfg["vocab"], D), "head": (cfg["vocab"], D), "final.norm": (D,)}
    for i, l in enumerate(cfg["layers"]):
        p, m, mx = "l%d." % i, "l%d.mix." % i, l["mixer"]
        H, ow = mx["heads"], mx["heads"] * mx["vdim"]
        out.update({p + "norm1": (D,), p + "ls1": (D,), m + "g": (ow if l["type"] == "delta" else H, D), m + "o": (D, ow)})
        if l["type"] == "delta":
            nq = mx["kv_heads"] * mx["dim"]
            for n, rows in (("q", nq), ("k", nq), ("v", ow)):
                out[m + n], out[m + n + ".conv"] = (rows, D), (rows, mx["conv"])
            out.update({m + "b": (H, D), m + "a": (H, D), m + "A_log": (H,), m + "dt_bias": (H,), m + "norm": (mx["vdim"],)})
        else:
            r, k, d = mx["q_rank"], mx["kv_rank"], mx["dim"]
            out.update({m + "dq": (r, D), m + "dq.norm": (r,), m + "uq": (H * (d + mx["rot_dim"]), r),
                        m + "uk": (H * d, k), m + "uv": (H * mx["vdim"], k)})
            if "kv_from" not in mx:
                out.update({m + "dkv": (k + mx["rot_dim"], D), m + "dkv.norm": (k,)})
        if l["mlp"]:
            f, ff = p + "mlp.", l["mlp"]["ff"]
            out.update({p + "norm2": (D,), p + "ls2": (D,), f + "gate": (ff, D), f + "up": (ff, D), f + "down": (D, ff)})
    return out


def weights(cfg, seed=0):
    """Random weights of a size that makes every mechanism count: decays between almost none and strong, clamps that
    bite, attention that is not flat."""
    rng = np.random.default_rng(seed)
    w = {}
    for name, shape in sorted(shapes(cfg).items()):
        leaf = name.split(".")[-1]
        if leaf == "A_log":
            a = np.log(rng.uniform(0.02, 4.0, shape))
        elif leaf == "dt_bias":
            a = rng.uniform(-3.0, 0.5, shape)
        elif leaf == "conv":
            a = rng.normal(0, 0.6, shape)
        elif "norm" in leaf:
            a = 1.0 + 0.3 * rng.normal(size=shape)
        elif leaf == "correction":
            a = 0.15 * rng.normal(size=shape) - 0.1
        elif leaf in ("ls1", "ls2"):
            a = rng.uniform(0.3, 1.2, shape) * rng.choice([-1.0, 1.0], shape)
        elif leaf == "embed" or len(shape) == 1:               # also the projections' biases
            a = rng.normal(size=shape)
        elif leaf in ("uq", "uk", "gate", "up", "b"):
            a = rng.normal(size=shape) * 2.0 / np.sqrt(shape[1])
        else:
            a = rng.normal(size=shape) * 1.5 / np.sqrt(shape[1])
        w[name] = bf16_round(a.astype(np.float32))
    return w


def tokens(cfg, n, seed=0):
    return [int(t) for t in np.random.default_rng(1000 + seed).integers(0, cfg["vocab"], n)]


def make_decoder(ops, cfg, w, dtype="float32", max_tokens=512, max_batch=4, state_slots=None, block_size=16, as_bf16=True):
    from fandhe_ai_amd import models
    from fandhe_ai_amd.safetensors_io import TypedTensor
    d = models.build_layered(ops, cfg, dtype, models.Capacity(max_tokens, max_batch, state_slots, block_size), shapes(cfg))
    typed = {}
    for n, a in w.items():
        if as_bf16:
            typed[n] = TypedTensor("BF16", a.shape, (a.view(np.uint32) >> 16).astype(np.uint16))
        else:
            typed[n] = TypedTensor("F32", a.shape, a)
    models.install_weights(d, typed)
    return d


def decided(cfg, w, toks, least=0.05):
    """The oracle's logits, and which positions' experts are no close calls (a rounding cannot change them)."""
    margins = []
    want = oracle.forward(cfg, w, toks, margins=margins)
    return want, np.min(margins + [np.full(len(toks), np.inf)], axis=0) >= least


def error(got, want):
    """Largest over the positions of the r.m.s. difference relative to the logits' overall r.m.s. (means taken off)."""
    got, want = np.asarray(got, np.float64), np.asarray(want, np.float64)
    d = got - want
    d -= d.mean(axis=-1, keepdims=True)
    c = want - want.mean(axis=-1, keepdims=True)
    return float(np.sqrt((d * d).mean(axis=-1)).max() / np.sqrt((c * c).mean()))
