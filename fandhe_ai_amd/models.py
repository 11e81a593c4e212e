"""Model registry: a folder with config.json and model.safetensors -> a resident decoder.

``load_model`` picks the design by config.json: its "architecture" (or the first of "architectures") names an entry of
``ARCHITECTURES``.  A new design registers a function that reads its configuration and weights and returns a decoder;
what the decoder runs on (pages, rows, state slots) is the caller's ``Capacity``.
"""
import json
import os
import re

from . import capi
from . import safetensors_io as st
from .decoder import LayeredDecoder

CONFIG_FILE, WEIGHTS_FILE = "config.json", "model.safetensors"


class ConfigError(ValueError):
    """A configuration that is incomplete or asks for something the framework does not have."""


class Capacity:
    """What a decoder is built to hold: ``max_tokens`` cached tokens over all sequences (whole pages), ``max_batch``
    sequences per step and ``state_slots`` recurrent states (default: one per row of the batch)."""

    def __init__(self, max_tokens, max_batch=32, state_slots=None, block_size=16):
        if min(max_tokens, max_batch, block_size) < 1:
            raise ConfigError("Capacity: sizes must be positive")
        self.max_tokens, self.max_batch, self.block_size = max_tokens, max_batch, block_size
        self.state_slots = max_batch if state_slots is None else state_slots

    @property
    def num_blocks(self):
        return -(-self.max_tokens // self.block_size)


DTYPES = {"bfloat16": capi.BF16, "float32": capi.F32}

# architecture name -> function(ops, config, weights path, dtype name, capacity) -> decoder
ARCHITECTURES = {}


def register(name):
    def add(fn):
        ARCHITECTURES[name] = fn
        return fn
    return add


def read_config(folder):
    try:
        with open(os.path.join(folder, CONFIG_FILE)) as f:
            return json.load(f)
    except (OSError, ValueError) as e:
        raise ConfigError("%s: %s" % (CONFIG_FILE, e))


def architecture_of(config):
    name = config.get("architecture") or (config.get("architectures") or [None])[0]
    if name not in ARCHITECTURES:
        raise ConfigError("unknown architecture %r (known: %s)" % (name, ", ".join(sorted(ARCHITECTURES))))
    return name


def load_model(ops, folder, dtype="bfloat16", capacity=None):
    """The decoder of the model in ``folder`` on ``ops``."""
    if dtype not in DTYPES:
        raise ConfigError("dtype must be one of %s" % ", ".join(sorted(DTYPES)))
    config = read_config(folder)
    build = ARCHITECTURES[architecture_of(config)]
    return build(ops, config, os.path.join(folder, WEIGHTS_FILE), dtype, capacity or Capacity(8192))


# ---- Nugelix: layers of gated delta rule and latent attention ---------------------------------------------------

GLU_ALPHA = 1.702                                          # the feed-forward's gate is g * sigmoid(1.702 g)


def _entry(d, key, where):
    if key not in d:
        raise ConfigError("%s: %r is missing" % (where, key))
    return d[key]


def nugelix_layers(config):
    """config.json's layer list as ``capi.LayerConfig`` fields."""
    out = []
    for i, layer in enumerate(_entry(config, "layers", CONFIG_FILE)):
        where = "layer %d" % i
        kind, mx = _entry(layer, "type", where), _entry(layer, "mixer", where)
        get = lambda key: _entry(mx, key, where + " mixer")
        l = {"heads": get("heads"), "dim": get("dim"), "vdim": get("vdim"), "kv_from": -1}
        if kind == "delta":
            l.update(mixer=capi.MIXER_DELTA, kv_heads=get("kv_heads"), conv=get("conv"))
        elif kind == "latent_attention":
            rot = get("rot")
            if _entry(rot, "dims", where + " rot") != get("rot_dim"):
                raise ConfigError("%s: all of the rotated part is rotated, rot.dims must equal rot_dim" % where)
            l.update(mixer=capi.MIXER_LATENT_ATTENTION, q_rank=get("q_rank"), kv_rank=get("kv_rank"), rot_dim=get("rot_dim"),
                     window=_entry(get("mask"), "size", where + " mask"), scale=get("scale"),
                     rot_base=_entry(rot, "base", where + " rot"))
            if mx.get("kv_from") is not None:
                l["kv_from"] = mx["kv_from"]
        else:
            raise ConfigError("%s: unknown type %r" % (where, kind))
        mlp = layer.get("mlp")
        if mlp is not None:
            if _entry(mlp, "kind", where + " mlp") != "dense":
                raise ConfigError("%s: unknown feed-forward %r" % (where, mlp["kind"]))
            l.update(d_ffn=_entry(mlp, "ff", where + " mlp"), ffn_limit=_entry(mlp, "limit", where + " mlp"), ffn_alpha=GLU_ALPHA)
        out.append(l)
    return out


def nugelix(config):
    """A Nugelix configuration as ``LayeredDecoder`` arguments."""
    return {"d_model": _entry(config, "width", CONFIG_FILE), "vocab": _entry(config, "vocab", CONFIG_FILE), "layers": nugelix_layers(config),
            "norm_eps": _entry(_entry(config, "norm", CONFIG_FILE), "eps", "norm"), "logit_softcap": config.get("logit_softcap") or 0.0}


# ---- Zoferax: grouped-query attention and sparse experts, sublayers normed at their output ------------------------

POSITION_BASE = 10000.0                                    # wavelengths of the additive positions


def zoferax_layers(config):
    """config.json's layer list as ``capi.LayerConfig`` fields."""
    out = []
    for i, layer in enumerate(_entry(config, "layers", CONFIG_FILE)):
        where = "layer %d" % i
        kind, mx = _entry(layer, "type", where), _entry(layer, "mixer", where)
        if kind != "attention":
            raise ConfigError("%s: unknown type %r" % (where, kind))
        l = {key: _entry(mx, key, where + " mixer") for key in ("heads", "kv_heads", "dim", "vdim", "scale")}
        l.update(mixer=capi.MIXER_ATTENTION, attention=capi.ATTENTION_BIAS | capi.ATTENTION_QK_NORM, kv_from=-1)
        if mx.get("kv_from") is not None:
            l["kv_from"] = mx["kv_from"]
        mlp = layer.get("mlp")
        if mlp is not None:
            if _entry(mlp, "kind", where + " mlp") != "moe":
                raise ConfigError("%s: unknown feed-forward %r" % (where, mlp["kind"]))
            router = _entry(mlp, "router", where + " mlp")
            l.update(d_ffn=_entry(_entry(mlp, "expert", where + " mlp"), "ff", where + " expert"),
                     experts=_entry(router, "experts", where + " router"), top=_entry(router, "top", where + " router"))
        out.append(l)
    return out


def zoferax(config):
    """A Zoferax configuration as ``LayeredDecoder`` arguments."""
    return {"d_model": _entry(config, "width", CONFIG_FILE), "vocab": _entry(config, "vocab", CONFIG_FILE), "layers": zoferax_layers(config),
            "norm_eps": _entry(_entry(config, "norm", CONFIG_FILE), "eps", "norm"), "logit_softcap": 0.0, "norm": capi.NORM_OUTPUT,
            "embed_scale": _entry(_entry(config, "embedding", CONFIG_FILE), "scale", "embedding"), "position_base": POSITION_BASE}


# ---- Bubetar: attention beside a recurrence, latent attention; sublayers normed on both sides ---------------------

def _rotation(mx, where, interleaved):
    """The rotation of a mixer's queries and keys as ``capi.LayerConfig`` fields."""
    rot = _entry(mx, "rot", where)
    out = {"rot_dim": _entry(rot, "dims", where + " rot"), "rot_base": _entry(rot, "base", where + " rot"), "rot_interleaved": int(interleaved)}
    if rot.get("scaling"):
        for key in ("factor", "low", "high", "original"):
            out["rot_" + key] = _entry(rot["scaling"], key, where + " rot scaling")
    return out


def _attention(mx, where, flags, interleaved):
    l = {key: _entry(mx, key, where) for key in ("heads", "kv_heads", "dim", "vdim", "scale")}
    l.update(_rotation(mx, where, interleaved), mixer=capi.MIXER_ATTENTION, attention=flags, kv_from=-1)
    if mx.get("mask"):
        l["window"] = _entry(mx["mask"], "size", where + " mask")
    return l


def _lightning(mx, where):
    l = {key: _entry(mx, key, where) for key in ("heads", "dim", "vdim", "decay")}
    if len(l["decay"]) != l["heads"]:
        raise ConfigError("%s: one decay per head" % where)
    return dict(l, mixer=capi.MIXER_LIGHTNING, kv_from=-1)


def _channel_delta(mx, where, prefix, shapes):
    """The ranks of the decays' and gates' projections are their weights' own."""
    l = {key: _entry(mx, key, where) for key in ("heads", "kv_heads", "dim", "vdim", "conv")}
    for field, name in (("decay_rank", prefix + "a1"), ("gate_rank", prefix + "g1")):
        if name not in shapes:
            raise ConfigError("%s: tensor %s is missing" % (where, name))
        l[field] = shapes[name][0]
    return dict(l, mixer=capi.MIXER_DELTA, kv_from=-1)


def bubetar_layers(config, shapes):
    """config.json's layer list as ``capi.LayerConfig`` fields; shapes: of the weights."""
    out = []
    for i, layer in enumerate(_entry(config, "layers", CONFIG_FILE)):
        where = "layer %d" % i
        kind, mx = _entry(layer, "type", where), _entry(layer, "mixer", where)
        at = where + " mixer"
        if kind in ("parallel", "parallel_2"):
            left, right = _entry(mx, "left", at), _entry(mx, "right", at)
            if kind == "parallel":
                l = _attention(left, at + " left", capi.ATTENTION_HEAD_NORM | capi.ATTENTION_GATE, True)
                r = _lightning(right, at + " right")
            else:
                l = _attention(left, at + " left", capi.ATTENTION_HEAD_UNIT | capi.ATTENTION_KEY_VALUES | capi.ATTENTION_SINK, False)
                r = _channel_delta(right, at + " right", "l%d.mix.right." % i, shapes)
            l.update(right=r, left_scale=_entry(mx, "left_scale", at), right_scale=_entry(mx, "right_scale", at))
        elif kind == "latent_attention":
            l = {key: _entry(mx, key, at) for key in ("heads", "dim", "vdim", "q_rank", "kv_rank", "scale")}
            l.update(_rotation(mx, at, True), mixer=capi.MIXER_LATENT_ATTENTION, ungated=1, kv_from=-1)
            if l["rot_dim"] != _entry(mx, "rot_dim", at):
                raise ConfigError("%s: all of the rotated part is rotated, rot.dims must equal rot_dim" % at)
        else:
            raise ConfigError("%s: unknown type %r" % (where, kind))
        mlp = layer.get("mlp")
        if mlp is not None:
            if _entry(mlp, "kind", where + " mlp") != "dense":
                raise ConfigError("%s: unknown feed-forward %r" % (where, mlp["kind"]))
            l.update(d_ffn=_entry(mlp, "ff", where + " mlp"), glu=capi.GLU_SILU)
        out.append(l)
    return out


def bubetar(config, shapes):
    """A Bubetar configuration as ``LayeredDecoder`` arguments."""
    scale = config.get("logit_scale")
    return {"d_model": _entry(config, "width", CONFIG_FILE), "vocab": _entry(config, "vocab", CONFIG_FILE), "layers": bubetar_layers(config, shapes),
            "norm_eps": _entry(_entry(config, "norm", CONFIG_FILE), "eps", "norm"), "norm": capi.NORM_BOTH,
            "logit_softcap": config.get("logit_softcap") or 0.0, "logit_scale": 1.0 if scale is None else scale}


# ---- Lugipel: minimal gated recurrences and windowed sigmoid attention, dense xIELU or sparse feed-forwards --------

DISTANCE_SPAN = 8.0                                        # slopes of the distance bias fall to 2^-8 over the heads


def _mingru(mx, where):
    return {"mixer": capi.MIXER_MINGRU, "heads": 1, "dim": 1, "vdim": _entry(mx, "width", where), "kv_from": -1}


def _sigmoid_attention(mx, where):
    l = {key: _entry(mx, key, where) for key in ("heads", "kv_heads", "dim", "vdim", "scale")}
    l.update(mixer=capi.MIXER_ATTENTION, attention=capi.ATTENTION_HEAD_NORM | capi.ATTENTION_SIGMOID | capi.ATTENTION_HEAD_GATE, kv_from=-1,
             distance=DISTANCE_SPAN)
    if mx.get("mask") is not None:
        l["window"] = _entry(mx["mask"], "size", where + " mask")
    if mx.get("q_temp") is not None:
        every = _entry(mx["q_temp"], "every", where + " q_temp")
        if every != int(every) or every < 1:
            raise ConfigError("%s: q_temp.every must be a positive whole number" % where)
        l.update(q_temp=_entry(mx["q_temp"], "coef", where + " q_temp"), q_temp_every=int(every))
    return l


def _scored_experts(mlp, where):
    """SiLU GLU experts chosen by scores, some of whose router outputs return the input."""
    router = _entry(mlp, "router", where)
    identity, at = router.get("identity") or 0, where + " router"
    l = {"d_ffn": _entry(_entry(mlp, "expert", where), "ff", where + " expert"), "experts": _entry(router, "experts", at) + identity,
         "identity": identity, "top": _entry(router, "top", at), "glu": capi.GLU_SILU, "route": capi.ROUTE_SCORED,
         "route_scale": _entry(router, "scale", at)}
    if router.get("groups") is not None:
        l.update(groups=_entry(router["groups"], "count", at + " groups"), groups_kept=_entry(router["groups"], "keep", at + " groups"))
    return l


def lugipel_layers(config):
    """config.json's layer list as ``capi.LayerConfig`` fields."""
    out, mixers = [], {"mingru": _mingru, "attention": _sigmoid_attention}
    for i, layer in enumerate(_entry(config, "layers", CONFIG_FILE)):
        where = "layer %d" % i
        kind, mlp = _entry(layer, "type", where), layer.get("mlp")
        if kind not in mixers:
            raise ConfigError("%s: unknown type %r" % (where, kind))
        l = mixers[kind](_entry(layer, "mixer", where), where + " mixer")
        if mlp is not None:
            ff = _entry(mlp, "kind", where + " mlp")
            if ff == "dense":
                l.update(d_ffn=_entry(mlp, "ff", where + " mlp"), glu=capi.FFN_XIELU)
            elif ff == "moe":
                l.update(_scored_experts(mlp, where + " mlp"))
            else:
                raise ConfigError("%s: unknown feed-forward %r" % (where, ff))
        out.append(l)
    return out


def lugipel(config):
    """A Lugipel configuration as ``LayeredDecoder`` arguments."""
    return {"d_model": _entry(config, "width", CONFIG_FILE), "vocab": _entry(config, "vocab", CONFIG_FILE), "layers": lugipel_layers(config),
            "norm_eps": _entry(_entry(config, "norm", CONFIG_FILE), "eps", "norm"), "logit_softcap": 0.0, "norm": capi.NORM_INPUT_RMS,
            "embed_scale": _entry(_entry(config, "embedding", CONFIG_FILE), "scale", "embedding"), "position_base": POSITION_BASE}


# designs made of described layers: architecture name -> function(config, shapes of the weights) -> LayeredDecoder arguments
LAYERED = {"Nugelix": lambda config, shapes: nugelix(config), "Zoferax": lambda config, shapes: zoferax(config), "Bubetar": bubetar,
           "Lugipel": lambda config, shapes: lugipel(config)}


def build_layered(ops, config, dtype, capacity, shapes=None):
    """The layered decoder a configuration describes, without weights.  shapes: tensor name -> shape, for designs some of whose
    sizes only the weights tell."""
    return LayeredDecoder(ops, max_blocks_per_seq=capacity.num_blocks, num_blocks=capacity.num_blocks, max_batch=capacity.max_batch,
                          state_slots=capacity.state_slots, dtype=DTYPES[dtype], block_size=capacity.block_size,
                          **LAYERED[architecture_of(config)](config, shapes or {}))


def install_weights(decoder, typed):
    """name -> ``safetensors_io.TypedTensor`` into a layered decoder: every tensor it takes, none it does not (norms of a
    feed-forward that a layer has not are passed over)."""
    wanted = decoder.tensors()
    st.require_keys(typed, sorted(wanted))
    extra = sorted(n for n in set(typed) - set(wanted) if not re.fullmatch(r"l\d+\.norm2b?", n))
    if extra:
        raise ConfigError("tensors the configuration has no use for: %s" % ", ".join(extra))
    for name, shape in wanted.items():
        t = typed[name]
        if t.shape != shape:
            raise st.SafetensorsFormat("%s has shape %s, the configuration needs %s" % (name, t.shape, shape))
        if t.dtype == "BF16":
            decoder.set_tensor(name, t.data, bf16=True)
        else:
            decoder.set_tensor(name, t.to_f32())


@register("Nugelix")
@register("Zoferax")
@register("Bubetar")
@register("Lugipel")
def _layered(ops, config, weights, dtype, capacity):
    typed = st.load_safetensors_typed(weights)
    decoder = build_layered(ops, config, dtype, capacity, {n: t.shape for n, t in typed.items()})
    try:
        install_weights(decoder, typed)
    except Exception:
        decoder.close()
        raise
    return decoder


# ---- Llama-style checkpoints on the W8A8 decoder ------------------------------------------------------------------

@register("LlamaForCausalLM")
def _llama(ops, config, weights, dtype, capacity):
    if dtype != "bfloat16":
        raise ConfigError("the W8A8 decoder has no float32 form")
    heads, get = _entry(config, "num_attention_heads", CONFIG_FILE), config.get
    decoder, store = st.load_decoder(ops, weights, _entry(config, "num_hidden_layers", CONFIG_FILE), heads,
                                     get("num_key_value_heads") or heads, capacity.num_blocks, capacity.num_blocks,
                                     min(capacity.max_batch, 64), get("head_dim") or config["hidden_size"] // heads, capacity.block_size,
                                     get("rms_norm_eps") or 1e-5, get("rope_theta") or 10000.0)
    ops.synchronize_device()
    store.free()
    return decoder
