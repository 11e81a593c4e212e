"""Oracle: the mechanisms of the layered decoders (gated delta rule, latent attention, clamped GLU feed-forward,
layer norm with layer scale, soft-capped head; grouped-query attention with normed projections, sparse experts, additive
positions, norms on the sublayers' outputs; two mixers side by side, rotations of either layout with scaled frequencies, norms
per head, output gates, sinks, lightning attention, the delta rule with a decay per channel, norms on both sides of a
sublayer; minimal gated recurrence, attention with sigmoid weights, distance biases, query temperature and gates per head, xIELU
feed-forward, experts in groups with identity experts), one function per mechanism, in float64 and token by token.

TEST INFRASTRUCTURE ONLY: written from the equations, for whole sequences, without a cache, a batch or any code
of the product; only tests and the smoke check may import it.

``weights`` maps tensor names to arrays (linear weights [out, in]); ``config`` is the parsed config.json.
"""
import numpy as np


def sigmoid(z):
    return 0.5 * (1.0 + np.tanh(0.5 * z))


def silu(z):
    return z * sigmoid(z)


def softplus(z):
    return np.maximum(z, 0.0) + np.log1p(np.exp(-np.abs(z)))


def rms_norm(x, w, eps):
    return x / np.sqrt((x * x).mean(axis=-1, keepdims=True) + eps) * w


def layer_norm(x, w, eps):
    c = x - x.mean(axis=-1, keepdims=True)
    return c / np.sqrt((c * c).mean(axis=-1, keepdims=True) + eps) * w


def unit_vector(x):
    return x / np.sqrt((x * x).sum(axis=-1, keepdims=True) + 1e-6)


def rotate(x, positions, base):
    """Rotate-half rotary embedding of all of x's last axis; positions has x's first axis."""
    dims = x.shape[-1]
    half = dims // 2
    freq = float(base) ** (-2.0 * np.arange(half) / dims)
    a = np.asarray(positions, dtype=np.float64)[:, None] * freq
    a = a.reshape((a.shape[0],) + (1,) * (x.ndim - 2) + (half,))
    u, v = x[..., :half], x[..., half:]
    return np.concatenate([u * np.cos(a) - v * np.sin(a), v * np.cos(a) + u * np.sin(a)], axis=-1)


def causal_conv(x, taps):
    """y_t = sum_i taps[:, i] x_{t - (T - 1) + i} per channel; zeros before the start."""
    n, T = x.shape[0], taps.shape[1]
    padded = np.concatenate([np.zeros((T - 1, x.shape[1])), x])
    return sum(padded[i:i + n] * taps[:, i] for i in range(T))


def delta_recurrence(q, k, v, beta, log_g):
    """q, k [T, H, dk] (k a unit vector), v [T, H, dv], beta / log_g [T, H] -> [T, H, dv]; the read-out follows
    the write."""
    T, H, dk = q.shape
    S = np.zeros((H, dk, v.shape[2]))
    out = np.empty_like(v)
    for t in range(T):
        S *= np.exp(log_g[t])[:, None, None]
        u = beta[t][:, None] * (v[t] - np.einsum("hkv,hk->hv", S, k[t]))
        S += k[t][:, :, None] * u[:, None, :]
        out[t] = np.einsum("hkv,hk->hv", S, q[t])
    return out


def delta_mixer(h, w, p, mx, eps):
    """The gated delta rule layer; p is the tensor prefix, mx its configuration entry."""
    T = h.shape[0]
    dim, vdim, heads, kvh = mx["dim"], mx["vdim"], mx["heads"], mx["kv_heads"]
    q, k, v = (silu(causal_conv(h @ w[p + n].T, w[p + n + ".conv"])) for n in "qkv")
    share = heads // kvh
    q = np.repeat(unit_vector(q.reshape(T, kvh, dim)), share, axis=1) * dim ** -0.5
    k = np.repeat(unit_vector(k.reshape(T, kvh, dim)), share, axis=1)
    beta = sigmoid(h @ w[p + "b"].T)
    log_g = -np.exp(w[p + "A_log"]) * softplus(h @ w[p + "a"].T + w[p + "dt_bias"])
    o = delta_recurrence(q, k, v.reshape(T, heads, vdim), beta, log_g)
    o = rms_norm(o, w[p + "norm"], eps) * silu(h @ w[p + "g"].T).reshape(T, heads, vdim)
    return o.reshape(T, heads * vdim) @ w[p + "o"].T


def latent_rows(h, w, p, mx, eps):
    """What a layer with a W_dkv of its own keeps of a token: the normed latent and the rotated shared key part."""
    y = h @ w[p + "dkv"].T
    r = mx["kv_rank"]
    return rms_norm(y[:, :r], w[p + "dkv.norm"], eps), rotate(y[:, r:], np.arange(len(h)), mx["rot"]["base"])


def windowed_softmax_attention(q, k, v, scale, window):
    """q, k [T, H, d], v [T, H, dv]; position i sees j with 0 <= i - j < window."""
    T = q.shape[0]
    i, j = np.arange(T)[:, None], np.arange(T)[None, :]
    seen = (j <= i) & (i - j < window)
    out = np.empty(v.shape)
    for h in range(q.shape[1]):
        s = np.where(seen, (q[:, h] @ k[:, h].T) * scale, -np.inf)
        s = np.exp(s - s.max(axis=1, keepdims=True))
        out[:, h] = (s / s.sum(axis=1, keepdims=True)) @ v[:, h]
    return out


def latent_mixer(h, kept, w, p, mx, eps):
    """Latent attention over kept = (latents, rotated key parts), which may be another layer's."""
    T = h.shape[0]
    H, dim, rot, vdim = mx["heads"], mx["dim"], mx["rot_dim"], mx["vdim"]
    c, kr = kept
    q = (rms_norm(h @ w[p + "dq"].T, w[p + "dq.norm"], eps) @ w[p + "uq"].T).reshape(T, H, dim + rot)
    q = np.concatenate([q[..., :dim], rotate(q[..., dim:], np.arange(T), mx["rot"]["base"])], axis=-1)
    k = (c @ w[p + "uk"].T).reshape(T, H, dim)
    k = np.concatenate([k, np.repeat(kr[:, None, :], H, axis=1)], axis=-1)
    v = (c @ w[p + "uv"].T).reshape(T, H, vdim)
    o = windowed_softmax_attention(q, k, v, mx["scale"], mx["mask"]["size"])
    o = o * sigmoid(h @ w[p + "g"].T)[:, :, None]
    return o.reshape(T, H * vdim) @ w[p + "o"].T


def clamped_glu(h, w, p, limit):
    g = np.minimum(h @ w[p + "gate"].T, limit)
    u = np.clip(h @ w[p + "up"].T, -limit, limit)
    return (g * sigmoid(1.702 * g) * (u + 1.0)) @ w[p + "down"].T


def softcap(z, cap):
    return cap * np.tanh(z / cap)


def sinusoid(positions, width):
    """Additive positions: sine in the even entries, cosine in the odd ones, of wavelengths growing to 10000 x 2 pi."""
    out = np.empty((len(positions), width))
    for e in range(width):
        a = np.asarray(positions, dtype=np.float64) * 10000.0 ** (-(e - e % 2) / width)
        out[:, e] = np.cos(a) if e % 2 else np.sin(a)
    return out


def grouped_kv(h, w, p, mx, eps):
    """What an attention layer with projections of its own keeps of every token: normed keys [T, G, dim], values
    [T, G, vdim].  The norm runs over the keys of all heads at once."""
    G = mx["kv_heads"]
    k = rms_norm(h @ w[p + "k"].T + w[p + "k.b"], w[p + "k.norm"], eps)
    v = h @ w[p + "v"].T + w[p + "v.b"]
    return k.reshape(len(h), G, mx["dim"]), v.reshape(len(h), G, mx["vdim"])


def grouped_attention(q, k, v, scale):
    """q [T, H, d], k [T, G, d], v [T, G, dv]: causal softmax attention, consecutive query heads sharing a key head."""
    share = q.shape[1] // k.shape[1]
    return windowed_softmax_attention(q, np.repeat(k, share, axis=1), np.repeat(v, share, axis=1), scale, len(q))


def grouped_mixer(h, kept, w, p, mx, eps):
    """The attention layer over kept = (keys, values), which may be another layer's."""
    q = rms_norm(h @ w[p + "q"].T + w[p + "q.b"], w[p + "q.norm"], eps)
    o = grouped_attention(q.reshape(len(h), mx["heads"], mx["dim"]), kept[0], kept[1], mx["scale"])
    return o.reshape(len(h), -1) @ w[p + "o"].T


def route(z, top):
    """Router logits [T, experts] -> weights [T, experts]: a softmax over the `top` largest, zero elsewhere."""
    out = np.zeros_like(z)
    for t, row in enumerate(z):
        best = np.argsort(-row, kind="stable")[:top]
        e = np.exp(row[best] - row[best].max())
        out[t, best] = e / e.sum()
    return out


def squared_relu_expert(h, w, p):
    return np.maximum(h @ w[p + "up"].T, 0.0) ** 2 @ w[p + "down"].T


def route_margin(z, top):
    """How far every row's choice is from another one: the gap between the last chosen logit and the first left out,
    relative to the row's spread (inf where nothing is left out)."""
    if top == z.shape[1]:
        return np.full(len(z), np.inf)
    s = -np.sort(-z, axis=1)
    return (s[:, top - 1] - s[:, top]) / (z.std(axis=1) + 1e-30)


def sparse_experts(h, w, p, mlp, margins=None):
    z = h @ w[p + "router"].T
    g = route(z, mlp["router"]["top"])
    if margins is not None:
        margins.append(route_margin(z, mlp["router"]["top"]))
    y = np.zeros_like(h)
    for e in range(mlp["router"]["experts"]):
        rows = np.nonzero(g[:, e])[0]
        y[rows] += g[rows, e:e + 1] * squared_relu_expert(h[rows], w, p + "e%d." % e)
    return y


def forward_zoferax(config, w, tokens, layers_out=None, margins=None):
    """Embedding with additive positions; sublayers read the residual itself and their outputs are normed."""
    eps = config["norm"]["eps"]
    x = w["embed"][np.asarray(tokens, dtype=np.int64)] * config["embedding"]["scale"] + sinusoid(np.arange(len(tokens)), config["width"])
    kept = {}
    for i, layer in enumerate(config["layers"]):
        p, mx = "l%d." % i, layer["mixer"]
        src = mx.get("kv_from", i)
        if src == i:
            kept[i] = grouped_kv(x, w, p + "mix.", mx, eps)
        x = x + rms_norm(grouped_mixer(x, kept[src], w, p + "mix.", mx, eps), w[p + "norm1"], eps)
        if layer["mlp"] is not None:
            x = x + rms_norm(sparse_experts(x, w, p + "mlp.", layer["mlp"], margins), w[p + "norm2"], eps)
        if layers_out is not None:
            layers_out.append(x.copy())
    return rms_norm(x, w["final.norm"], eps) @ w["head"].T


# ---- Bubetar ---------------------------------------------------------------------------------------------------

def scaled_frequencies(freq, scaling):
    """Rotation frequencies stretched for long contexts: long waves are slowed down by the factor, short ones stay, with a
    ramp between the two wavelengths original / high and original / low."""
    out = np.empty_like(freq)
    for i, f in enumerate(freq):
        turns = scaling["original"] * f / (2.0 * np.pi)              # of the wave within the original context
        if turns > scaling["high"]:
            out[i] = f
        elif turns < scaling["low"]:
            out[i] = f / scaling["factor"]
        else:
            s = (turns - scaling["low"]) / (scaling["high"] - scaling["low"])
            out[i] = (1.0 - s) * f / scaling["factor"] + s * f
    return out


def rotate_leading(x, positions, rot, interleaved):
    """Rotates the first rot["dims"] entries of x's last axis; x [T, heads, d].  Pairs are neighbours (interleaved) or half the
    rotated part apart."""
    dims = rot["dims"]
    freq = float(rot["base"]) ** (-2.0 * np.arange(dims // 2) / dims)
    if rot.get("scaling"):
        freq = scaled_frequencies(freq, rot["scaling"])
    first = np.arange(0, dims, 2) if interleaved else np.arange(dims // 2)
    second = first + 1 if interleaved else first + dims // 2
    out = np.array(x)
    for t, p in enumerate(positions):
        turn = np.exp(1j * p * freq)
        z = (x[t][:, first] + 1j * x[t][:, second]) * turn
        out[t][:, first], out[t][:, second] = z.real, z.imag
    return out


def sink_attention(q, k, v, scale, window=None, sink=None):
    """Causal attention with shared key heads; window None: every earlier token.  sink [H]: a score without key and value."""
    T, H = q.shape[:2]
    share = H // k.shape[1]
    out = np.empty((T, H, v.shape[2]))
    for t in range(T):
        lo = 0 if window is None else max(0, t - window + 1)
        for h in range(H):
            s = k[lo:t + 1, h // share] @ q[t, h] * scale
            m = s.max() if sink is None else max(s.max(), sink[h])
            e = np.exp(s - m)
            total = e.sum() + (0.0 if sink is None else np.exp(sink[h] - m))
            out[t, h] = e @ v[lo:t + 1, h // share] / total
    return out


def gated_attention_mixer(h, w, p, mx, eps):
    """Normed, rotated queries and keys; the heads' outputs pass a gate read from the same input."""
    T, H, G, d = len(h), mx["heads"], mx["kv_heads"], mx["dim"]
    q = rms_norm((h @ w[p + "q"].T).reshape(T, H, d), w[p + "q.norm"], eps)
    k = rms_norm((h @ w[p + "k"].T).reshape(T, G, d), w[p + "k.norm"], eps)
    q, k = (rotate_leading(a, range(T), mx["rot"], True) for a in (q, k))
    o = sink_attention(q, k, (h @ w[p + "v"].T).reshape(T, G, mx["vdim"]), mx["scale"])
    return (o.reshape(T, -1) * sigmoid(h @ w[p + "g"].T)) @ w[p + "o"].T


def key_value_attention_mixer(h, w, p, mx, eps):
    """The projected keys are the values; queries and keys are rotated, then normed without a weight; window and sink."""
    T, H, G, d = len(h), mx["heads"], mx["kv_heads"], mx["dim"]
    q, k = (h @ w[p + "q"].T).reshape(T, H, d), (h @ w[p + "k"].T).reshape(T, G, d)
    qr, kr = (rms_norm(rotate_leading(a, range(T), mx["rot"], False), 1.0, eps) for a in (q, k))
    o = sink_attention(qr, kr, k, mx["scale"], mx["mask"]["size"], w[p + "sink"])
    return o.reshape(T, -1) @ w[p + "o"].T


def lightning_recurrence(q, k, v, decay):
    """S <- decay S + k v^T, o = S^T q per head; q, k [T, H, dk], v [T, H, dv]."""
    S = np.zeros((q.shape[1], q.shape[2], v.shape[2]))
    out = np.empty(v.shape)
    for t in range(len(q)):
        for h in range(len(S)):
            S[h] = decay[h] * S[h] + np.outer(k[t, h], v[t, h])
            out[t, h] = q[t, h] @ S[h]
    return out


def lightning_mixer(h, w, p, mx, eps):
    T, H = len(h), mx["heads"]
    q, k, v = (silu(h @ w[p + n].T).reshape(T, H, -1) for n in "qkv")
    o = lightning_recurrence(q, k, v, mx["decay"]).reshape(T, -1)
    return (rms_norm(o, w[p + "norm"], eps) * sigmoid(h @ w[p + "g"].T)) @ w[p + "o"].T


def channel_delta_recurrence(q, k, v, beta, log_g):
    """The delta rule with log decays [T, H, dk]: one per head and row of the state."""
    S = np.zeros((q.shape[1], q.shape[2], v.shape[2]))
    out = np.empty(v.shape)
    for t in range(len(q)):
        for h in range(len(S)):
            S[h] *= np.exp(log_g[t, h])[:, None]
            u = beta[t, h] * (v[t, h] - k[t, h] @ S[h])
            S[h] += np.outer(k[t, h], u)
            out[t, h] = q[t, h] @ S[h]
    return out


def channel_delta_mixer(h, w, p, mx, eps):
    T, dim, vdim, heads, kvh = len(h), mx["dim"], mx["vdim"], mx["heads"], mx["kv_heads"]
    q, k, v = (silu(causal_conv(h @ w[p + n].T, w[p + n + ".conv"])) for n in "qkv")
    own = np.arange(heads) // (heads // kvh)
    q = unit_vector(q.reshape(T, kvh, dim))[:, own] * dim ** -0.5
    k = unit_vector(k.reshape(T, kvh, dim))[:, own]
    beta = sigmoid(h @ w[p + "b"].T)
    a = softplus(h @ w[p + "a1"].T @ w[p + "a2"].T + w[p + "dt_bias"]).reshape(T, heads, dim)
    o = channel_delta_recurrence(q, k, v.reshape(T, heads, vdim), beta, -np.exp(w[p + "A_log"])[None, :, None] * a)
    o = rms_norm(o, w[p + "norm"], eps).reshape(T, -1) * sigmoid(h @ w[p + "g1"].T @ w[p + "g2"].T)
    return o @ w[p + "o"].T


def plain_latent_mixer(h, w, p, mx, eps):
    """Latent attention without a gate over all earlier tokens, the rotated parts in pairs of neighbours."""
    T, H, dim, r = len(h), mx["heads"], mx["dim"], mx["kv_rank"]
    q = (rms_norm(h @ w[p + "dq"].T, w[p + "dq.norm"], eps) @ w[p + "uq"].T).reshape(T, H, -1)
    y = h @ w[p + "dkv"].T
    c = rms_norm(y[:, :r], w[p + "dkv.norm"], eps)
    kr = rotate_leading(y[:, None, r:], range(T), mx["rot"], True)
    q = np.concatenate([q[..., :dim], rotate_leading(q[..., dim:], range(T), mx["rot"], True)], axis=-1)
    k = np.concatenate([(c @ w[p + "uk"].T).reshape(T, H, dim), np.repeat(kr, H, axis=1)], axis=-1)
    o = sink_attention(q, k, (c @ w[p + "uv"].T).reshape(T, H, -1), mx["scale"])
    return o.reshape(T, -1) @ w[p + "o"].T


def side_by_side(h, w, p, mx, eps, left, right):
    return mx["left_scale"] * left(h, w, p + "left.", mx["left"], eps) + mx["right_scale"] * right(h, w, p + "right.", mx["right"], eps)


def silu_glu(h, w, p):
    return (silu(h @ w[p + "gate"].T) * (h @ w[p + "up"].T)) @ w[p + "down"].T


def forward_bubetar(config, w, tokens, layers_out=None):
    """Every sublayer is normed on both sides; scaled, soft-capped logits."""
    eps = config["norm"]["eps"]
    x = w["embed"][np.asarray(tokens, dtype=np.int64)]
    for i, layer in enumerate(config["layers"]):
        p, mx = "l%d." % i, layer["mixer"]
        h = layer_norm(x, w[p + "norm1"], eps)
        if layer["type"] == "parallel":
            y = side_by_side(h, w, p + "mix.", mx, eps, gated_attention_mixer, lightning_mixer)
        elif layer["type"] == "parallel_2":
            y = side_by_side(h, w, p + "mix.", mx, eps, key_value_attention_mixer, channel_delta_mixer)
        else:
            y = plain_latent_mixer(h, w, p + "mix.", mx, eps)
        x = x + layer_norm(y, w[p + "norm1b"], eps)
        if layer["mlp"] is not None:
            x = x + layer_norm(silu_glu(layer_norm(x, w[p + "norm2"], eps), w, p + "mlp."), w[p + "norm2b"], eps)
        if layers_out is not None:
            layers_out.append(x.copy())
    return softcap(layer_norm(x, w["final.norm"], eps) @ w["head"].T * config["logit_scale"], config["logit_softcap"])


# ---- Lugipel ---------------------------------------------------------------------------------------------------

def gated_recurrence(z, candidate):
    """S <- (1 - z) S + z candidate, entry by entry; z, candidate [T, width] -> every S."""
    S = np.zeros(z.shape[1])
    out = np.empty_like(z)
    for t in range(len(z)):
        S = (1.0 - z[t]) * S + z[t] * candidate[t]
        out[t] = S
    return out


def positive_candidate(u):
    """u + 1/2 from zero on, the logistic function below: continuous and never negative."""
    return np.where(u >= 0.0, u + 0.5, sigmoid(np.minimum(u, 0.0)))


def mingru_mixer(h, w, p):
    """The recurrence's gates read the current token only."""
    z = sigmoid(h @ w[p + "z"].T + w[p + "z.b"])
    S = gated_recurrence(z, positive_candidate(h @ w[p + "x"].T + w[p + "x.b"]))
    return (S * silu(h @ w[p + "g"].T)) @ w[p + "o"].T


def query_temperature(positions, coef, every):
    """1 in the first `every` - 1 positions, growing with the logarithm of the number of whole blocks seen."""
    return np.array([1.0 + coef * np.log(float((p + 1) // every) + 1.0) for p in positions])


def distance_slopes(heads):
    """Geometric from 2^(-8 / heads) down to 2^-8."""
    return np.array([2.0 ** (-8.0 * (h + 1) / heads) for h in range(heads)])


def sigmoid_attention(q, k, v, scale, window, slopes, bias):
    """Weights sigmoid(q . k scale - slope (i - j) + bias), not normalized; position i sees the last `window` tokens."""
    T, H = q.shape[:2]
    share = H // k.shape[1]
    out = np.empty((T, H, v.shape[2]))
    for t in range(T):
        j = np.arange(0 if window is None else max(0, t - window + 1), t + 1)
        for h in range(H):
            s = k[j, h // share] @ q[t, h] * scale - slopes[h] * (t - j) + bias[h]
            out[t, h] = sigmoid(s) @ v[j, h // share]
    return out


def sigmoid_attention_mixer(h, w, p, mx, eps):
    T, H, G, d = len(h), mx["heads"], mx["kv_heads"], mx["dim"]
    q = rms_norm((h @ w[p + "q"].T).reshape(T, H, d), w[p + "q.norm"], eps)
    k = rms_norm((h @ w[p + "k"].T).reshape(T, G, d), w[p + "k.norm"], eps)
    if mx.get("q_temp"):
        q = q * query_temperature(range(T), mx["q_temp"]["coef"], mx["q_temp"]["every"])[:, None, None]
    window = mx["mask"]["size"] if mx.get("mask") else None
    o = sigmoid_attention(q, k, (h @ w[p + "v"].T).reshape(T, G, mx["vdim"]), mx["scale"], window, distance_slopes(H), w[p + "pb"])
    return (o * sigmoid(h @ w[p + "g"].T)[:, :, None]).reshape(T, -1) @ w[p + "o"].T


def xielu(z, p, q):
    n = np.minimum(z, 0.0)
    return np.where(z > 0.0, softplus(p) * z * z, (0.5 + softplus(q)) * (np.expm1(n) - n)) + 0.5 * z


def xielu_forward(h, w, p):
    return xielu(h @ w[p + "up"].T, *w[p + "act"]) @ w[p + "down"].T


def grouped_choice(s, correction, top, groups, keep):
    """The chosen experts of one row of scores, and how close the choice is: the least distance of a choice score, or of a
    group's, to one on the other side, relative to the scores' spread."""
    c = s + correction
    size, spread = len(c) // groups, s.std() + 1e-30
    best = c.reshape(groups, size).max(axis=1)
    order = np.argsort(-best, kind="stable")
    margin = best[order[keep - 1]] - best[order[keep]] if keep < groups else np.inf
    allowed = np.repeat(np.isin(np.arange(groups), order[:keep]), size)
    c = np.where(allowed, c, -np.inf)
    order = np.argsort(-c, kind="stable")
    if top < int(allowed.sum()):
        margin = min(margin, c[order[top - 1]] - c[order[top]])
    return order[:top], margin / spread


def route_scored(z, correction, router):
    """Router logits [T, outputs] -> weights [T, outputs] and choice margins [T]."""
    groups = router.get("groups") or {"count": 1, "keep": 1}
    out, margins = np.zeros_like(z), np.empty(len(z))
    for t, row in enumerate(z):
        e = np.exp(row - row.max())
        s = e / e.sum()
        best, margins[t] = grouped_choice(s, correction, router["top"], groups["count"], groups["keep"])
        out[t, best] = s[best] / (s[best].sum() + 1e-20) * router["scale"]
    return out, margins


def scored_experts(h, w, p, mlp, margins=None):
    """Sparse SiLU GLU experts; the last router outputs belong to experts that return their input."""
    router = mlp["router"]
    g, m = route_scored(h @ w[p + "router"].T, w[p + "correction"], router)
    if margins is not None:
        margins.append(m)
    n = router["experts"]
    y = g[:, n:].sum(axis=1, keepdims=True) * h
    for e in range(n):
        rows = np.nonzero(g[:, e])[0]
        y[rows] += g[rows, e:e + 1] * silu_glu(h[rows], w, p + "e%d." % e)
    return y


def forward_lugipel(config, w, tokens, layers_out=None, margins=None):
    """RMS norms ahead of every sublayer, additive positions."""
    eps = config["norm"]["eps"]
    x = w["embed"][np.asarray(tokens, dtype=np.int64)] * config["embedding"]["scale"] + sinusoid(np.arange(len(tokens)), config["width"])
    for i, layer in enumerate(config["layers"]):
        p, mx = "l%d." % i, layer["mixer"]
        h = rms_norm(x, w[p + "norm1"], eps)
        x = x + (mingru_mixer(h, w, p + "mix.") if layer["type"] == "mingru" else sigmoid_attention_mixer(h, w, p + "mix.", mx, eps))
        if layer["mlp"] is not None:
            h = rms_norm(x, w[p + "norm2"], eps)
            x = x + (xielu_forward(h, w, p + "mlp.") if layer["mlp"]["kind"] == "dense" else scored_experts(h, w, p + "mlp.", layer["mlp"], margins))
        if layers_out is not None:
            layers_out.append(x.copy())
    return rms_norm(x, w["final.norm"], eps) @ w["head"].T


def forward(config, weights, tokens, layers_out=None, margins=None):
    """Logits [T, vocab] of one whole sequence; layers_out (a list) receives the residual after every layer, margins (a
    list) the routing margins of every layer of sparse experts."""
    w = {n: np.asarray(a, dtype=np.float64) for n, a in weights.items()}
    if config["architecture"] == "Zoferax":
        return forward_zoferax(config, w, tokens, layers_out, margins)
    if config["architecture"] == "Lugipel":
        return forward_lugipel(config, w, tokens, layers_out, margins)
    if config["architecture"] == "Bubetar":
        return forward_bubetar(config, w, tokens, layers_out)
    eps = config["norm"]["eps"]
    x = w["embed"][np.asarray(tokens, dtype=np.int64)]
    kept = {}
    for i, layer in enumerate(config["layers"]):
        p, mx = "l%d." % i, layer["mixer"]
        h = layer_norm(x, w[p + "norm1"], eps)
        if layer["type"] == "delta":
            y = delta_mixer(h, w, p + "mix.", mx, eps)
        else:
            src = mx.get("kv_from", i)
            if src == i:
                kept[i] = latent_rows(h, w, p + "mix.", mx, eps)
            y = latent_mixer(h, kept[src], w, p + "mix.", mx, eps)
        x = x + y * w[p + "ls1"]
        if layer["mlp"] is not None:
            x = x + clamped_glu(layer_norm(x, w[p + "norm2"], eps), w, p + "mlp.", layer["mlp"]["limit"]) * w[p + "ls2"]
        if layers_out is not None:
            layers_out.append(x.copy())
    return softcap(layer_norm(x, w["final.norm"], eps) @ w["head"].T, config["logit_softcap"])
