"""Plain, slow statement of the layer-stack models in numpy double precision: Varasun (latent attention,
the channel-decay delta rule) and Lofudra (windowed attention beside retention, mLSTM, Mamba-2, a loop
over some of the layers), Fobanex (normed and gated attention, shared latents, mixtures) and Minodra (latent
attention without positions, gated sublayers behind short convolutions, mixtures with a corrected choice).

One function per mechanism, whole sequences only: no cache, no pages, no batches.  Nothing here is
shared with the product path; the tests compare the driver with it and plant their mistakes here.
Weights are a dict name -> float array under the checkpoint's tensor names.
"""
from __future__ import annotations

import math

import numpy as np


def rms_norm(x, w, eps):
    x = np.asarray(x, np.float64)
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps) * w


def unit_vector(x, eps=1e-6):
    return x / np.sqrt(np.sum(x * x, axis=-1, keepdims=True) + eps)


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def silu(z):
    return z * sigmoid(z)


def softplus(z):
    return np.logaddexp(0.0, z)


def squared_relu(z):
    return np.square(np.maximum(z, 0.0))


def gelu_erf(z):
    return 0.5 * z * (1.0 + np.vectorize(math.erf)(z / math.sqrt(2.0)))


def log_sigmoid(z):
    return -np.logaddexp(0.0, -z)


def divide_by_rms(x, eps):
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def rotation_frequencies(rot: dict):
    """(frequency per pair, factor on cos and sin) of a rotation spec {dims, base, scaling}."""
    dims, base = int(rot["dims"]), float(rot["base"])
    i = np.arange(dims // 2, dtype=np.float64)
    f = base ** (-2.0 * i / dims)
    sc = rot.get("scaling")
    if not sc:
        return f, 1.0

    def pair_with_turns(turns):
        return dims * math.log(sc["original"] / (2.0 * math.pi * turns)) / (2.0 * math.log(base))

    lo = max(math.floor(pair_with_turns(sc["fast"])), 0)
    hi = min(math.ceil(pair_with_turns(sc["slow"])), dims - 1)
    ramp = np.clip((i - lo) / max(hi - lo, 0.001), 0.0, 1.0)
    return f / sc["factor"] * ramp + f * (1.0 - ramp), 0.1 * math.log(sc["factor"]) + 1.0


def rotate_pairs(x, positions, rot: dict):
    """Interleaved rotation of the first rot['dims'] entries of the last axis; x is [T, ..., n]."""
    f, m = rotation_frequencies(rot)
    ang = np.asarray(positions, np.float64)[:, None] * f
    shape = (len(positions),) + (1,) * (x.ndim - 2) + (len(f),)
    c, s = (np.cos(ang) * m).reshape(shape), (np.sin(ang) * m).reshape(shape)
    out = np.array(x, np.float64)
    n = 2 * len(f)
    u, v = x[..., 0:n:2], x[..., 1:n:2]
    out[..., 0:n:2] = u * c - v * s
    out[..., 1:n:2] = v * c + u * s
    return out


def causal_conv(x, w):
    """y[t, c] = sum_j w[c, j] * x[t - (taps - 1) + j, c], zeros before the start."""
    taps = w.shape[1]
    pad = np.concatenate([np.zeros((taps - 1, x.shape[1])), x])
    return sum(pad[j:j + len(x)] * w[:, j] for j in range(taps))


def causal_softmax_attention(scores, values):
    """scores [H, T, T], values [T, H, dv] -> [T, H, dv]; row i sees columns j <= i."""
    T = scores.shape[1]
    s = np.where(np.tril(np.ones((T, T), bool)), scores, -np.inf)
    p = np.exp(s - s.max(axis=-1, keepdims=True))
    p /= p.sum(axis=-1, keepdims=True)
    return np.einsum("hij,jhd->ihd", p, values)


def latent_attention(h, w, p, m, eps):
    T = len(h)
    H, dim, rd, dv, rank = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    pos = np.arange(T)
    cq = rms_norm(h @ w[p + "dq"].T, w[p + "dq.norm"], eps)
    q = (cq @ w[p + "uq"].T).reshape(T, H, dim + rd)
    qn, qr = q[..., :dim], rotate_pairs(q[..., dim:], pos, m["rot"])
    kv = h @ w[p + "dkv"].T
    c = rms_norm(kv[:, :rank], w[p + "dkv.norm"], eps)
    kr = rotate_pairs(kv[:, rank:], pos, m["rot"])
    kn = (c @ w[p + "uk"].T).reshape(T, H, dim)
    v = (c @ w[p + "uv"].T).reshape(T, H, dv)
    scores = (np.einsum("ihd,jhd->hij", qn, kn) + np.einsum("ihd,jd->hij", qr, kr)) * m["scale"]
    return causal_softmax_attention(scores, v).reshape(T, H * dv) @ w[p + "o"].T


def decay_of(h, w, p, H, dim):
    raw = (h @ w[p + "a1"].T) @ w[p + "a2"].T + w[p + "dt_bias"]
    return np.exp(-np.exp(w[p + "A_log"])[:, None] * softplus(raw).reshape(len(h), H, dim))


def delta_rule(q, k, v, g, beta):
    """q, k, g [T, H, dk]; v [T, H, dv]; beta [T, H] -> read-outs [T, H, dv]."""
    T, H, dk = q.shape
    S = np.zeros((H, dk, v.shape[-1]))
    out = np.empty_like(v)
    for t in range(T):
        S = g[t][:, :, None] * S
        u = beta[t][:, None] * (v[t] - np.einsum("hkv,hk->hv", S, k[t]))
        S = S + k[t][:, :, None] * u[:, None, :]
        out[t] = np.einsum("hkv,hk->hv", S, q[t])
    return out


def channel_delta(h, w, p, m, eps):
    T = len(h)
    H, G, dk, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k, v = (silu(causal_conv(h @ w[p + n].T, w[p + n + ".conv"])) for n in "qkv")
    q = unit_vector(q.reshape(T, G, dk)) * dk ** -0.5
    k = unit_vector(k.reshape(T, G, dk))
    src = np.arange(H) // (H // G)
    beta = sigmoid(h @ w[p + "b"].T)
    o = delta_rule(q[:, src], k[:, src], v.reshape(T, H, dv), decay_of(h, w, p, H, dk), beta)
    gate = sigmoid((h @ w[p + "g1"].T) @ w[p + "g2"].T).reshape(T, H, dv)
    return (rms_norm(o, w[p + "norm"], eps) * gate).reshape(T, H * dv) @ w[p + "o"].T


def rotate_halves(x, positions, rot: dict):
    """Rotation of the first rot['dims'] entries, entry i with entry i + dims/2; x is [T, ..., n]."""
    n = int(rot["dims"])
    perm = np.arange(x.shape[-1])
    perm[0:n:2], perm[1:n:2] = np.arange(n // 2), np.arange(n // 2, n)
    out = np.empty_like(np.asarray(x, np.float64))
    out[..., perm] = rotate_pairs(np.asarray(x)[..., perm], positions, rot)
    return out


def window_mask(T, window):
    """[T, T]: row i sees itself and the window - 1 columns before it (None: all before it)."""
    d = np.arange(T)[:, None] - np.arange(T)[None, :]
    return (d >= 0) & (d < (window if window else T + 1))


def softmax_with_sink(scores, seen, sink=1.0):
    """Weights of the seen columns; `sink` is added to the sum of exponentials."""
    s = np.where(seen, scores, -np.inf)
    m = np.maximum(s.max(axis=-1, keepdims=True), 0.0)
    p = np.exp(s - m)
    return p / (p.sum(axis=-1, keepdims=True) + sink * np.exp(-m))


def window_attention(h, w, p, m, eps):
    """Grouped-query attention over a sliding window; the raw keys are the values."""
    T, H, G, dim = len(h), m["heads"], m["kv_heads"], m["dim"]
    q = (h @ w[p + "q"].T + w[p + "q.b"]).reshape(T, H, dim)
    k = (h @ w[p + "k"].T + w[p + "k.b"]).reshape(T, G, dim)
    src = np.arange(H) // (H // G)
    pos = np.arange(T)
    v = k[:, src]
    q = rotate_halves(rms_norm(q, w[p + "q.norm"], eps), pos, m["rot"])
    k = rotate_halves(rms_norm(k, w[p + "k.norm"], eps), pos, m["rot"])[:, src]
    a = softmax_with_sink(np.einsum("ihd,jhd->hij", q, k) * m["scale"], window_mask(T, m["mask"]["size"]))
    return np.einsum("hij,jhd->ihd", a, v).reshape(T, -1) @ w[p + "o"].T


def decayed_outer_products(q, k, v, decay):
    """S_t = decay_t S_(t-1) + k_t v_t^T, o_t = S_t^T q_t: q, k [T, H, dk], v [T, H, dv], decay [T, H]."""
    T, H, dk = q.shape
    S = np.zeros((H, dk, v.shape[-1]))
    out = np.empty(v.shape)
    for t in range(T):
        S = decay[t][:, None, None] * S + k[t][:, :, None] * v[t][:, None, :]
        out[t] = np.einsum("hkv,hk->hv", S, q[t])
    return out


def retention(h, w, p, m, eps):
    T, H, dk, dv = len(h), m["heads"], m["dim"], m["vdim"]
    q, k, v = (h @ w[p + n].T for n in "qkv")
    decay = np.broadcast_to(np.asarray(m["decay"], np.float64), (T, H))
    o = decayed_outer_products(q.reshape(T, H, dk), k.reshape(T, H, dk) * dk ** -0.5, v.reshape(T, H, dv), decay)
    return (divide_by_rms(o, eps).reshape(T, H * dv) * silu(h @ w[p + "g"].T)) @ w[p + "o"].T


def parallel(h, w, p, m, eps):
    return (m["left_scale"] * window_attention(h, w, p + "left.", m["left"], eps)
            + m["right_scale"] * retention(h, w, p + "right.", m["right"], eps))


def matrix_memory(q, k, v, i, f):
    """Exponential input gate i and log forget gate f [T, H] with a running maximum from 0; q is scaled."""
    T, H, dk = q.shape
    S, n, m = np.zeros((H, dk, v.shape[-1])), np.zeros((H, dk)), np.zeros(H)
    out = np.empty(v.shape)
    for t in range(T):
        m_new = np.maximum(f[t] + m, i[t])
        keep, write = np.exp(f[t] + m - m_new), np.exp(i[t] - m_new)
        S = keep[:, None, None] * S + write[:, None, None] * k[t][:, :, None] * v[t][:, None, :]
        n = keep[:, None] * n + write[:, None] * k[t]
        m = m_new
        out[t] = np.einsum("hkv,hk->hv", S, q[t]) / (np.maximum(np.abs((n * q[t]).sum(-1)), np.exp(-m)) + 1e-6)[:, None]
    return out


def mlstm(h, w, p, m, eps):
    T, H, dk, dv, cap = len(h), m["heads"], m["dim"], m["vdim"], m["gate_cap"]
    q, k, v = (h @ w[p + n].T for n in "qkv")
    i, f = (cap * np.tanh((h @ w[p + n].T + w[p + n + ".b"]) / cap) for n in "if")
    o = matrix_memory(q.reshape(T, H, dk) * dk ** -0.5, k.reshape(T, H, dk), v.reshape(T, H, dv), i, log_sigmoid(f))
    return (divide_by_rms(o, eps).reshape(T, H * dv) * w[p + "norm"] * sigmoid(h @ w[p + "g"].T)) @ w[p + "o"].T


def mamba2(h, w, p, m, eps):
    T, H, dv, N, G = len(h), m["heads"], m["vdim"], m["state"], m["groups"]
    inner = H * dv
    z, xbc, dt = np.split(h @ w[p + "in"].T, [inner, 2 * inner + 2 * G * N], axis=-1)
    x, B, C = np.split(silu(causal_conv(xbc, w[p + "conv"]) + w[p + "conv.b"]), [inner, inner + G * N], axis=-1)
    x, B, C = x.reshape(T, H, dv), B.reshape(T, G, N), C.reshape(T, G, N)
    src = np.arange(H) // (H // G)
    dt = softplus(dt + w[p + "dt_bias"])
    y = decayed_outer_products(C[:, src], B[:, src], dt[:, :, None] * x, np.exp(-np.exp(w[p + "A_log"]) * dt))
    y = (y + w[p + "D"][:, None] * x).reshape(T, inner) * silu(z)
    y = divide_by_rms(y.reshape(T, m["norm_groups"], -1), eps).reshape(T, inner) * w[p + "norm"]
    return y @ w[p + "o"].T


MIXERS = {"latent_attention": latent_attention, "channel_delta": channel_delta, "parallel": parallel, "mlstm": mlstm,
          "mamba2": mamba2}


def feed_forward(x, w, p):
    return squared_relu(x @ w[p + "up"].T) @ w[p + "down"].T


def gelu_feed_forward(x, w, p):
    return gelu_erf(x @ w[p + "up"].T) @ w[p + "down"].T


def layer_runs(cfg):
    """(layer, number of its pass, whether a looped pass begins here) in the order they are run."""
    n = len(cfg["layers"])
    loop = cfg.get("loop") or dict(start=n, stop=n, times=1)
    a, b = loop["start"], loop["stop"]
    looped = [(i, t, i == a) for t in range(loop["times"]) for i in range(a, b)]
    return [(i, 0, False) for i in range(a)] + looped + [(i, 0, False) for i in range(b, n)]


def forward_sandwich(cfg, w, tokens, want_layers=False):
    """Norms ahead of and after every sublayer, some layers run several times with the same weights."""
    eps = cfg["norm"]["eps"]
    e = np.asarray(w["embed"], np.float64)[np.asarray(tokens)]
    x, states = e, []
    for i, t, begins in layer_runs(cfg):
        layer, p = cfg["layers"][i], f"l{i}."
        if begins:
            x = x + (e if t > 0 else 0.0) + w["loop.step"][t]
        y = MIXERS[layer["type"]](rms_norm(x, w[p + "norm1"], eps), w, p + "mix.", layer["mixer"], eps)
        x = x + rms_norm(y, w[p + "norm1b"], eps)
        if layer.get("mlp"):
            y = gelu_feed_forward(rms_norm(x, w[p + "norm2"], eps), w, p + "mlp.")
            x = x + rms_norm(y, w[p + "norm2b"], eps)
        states.append(x)
    logits = rms_norm(x, w["final.norm"], eps) @ w["head"].T
    return (logits, np.stack(states)) if want_layers else logits


# ---- Fobanex ---------------------------------------------------------------------------------------
def grouped_attention(q, k, v, scale):
    """q [T, H, d], k [T, G, d], v [T, G, dv]; query head h reads key head h // (H / G) -> [T, H, dv]."""
    src = np.arange(q.shape[1]) // (q.shape[1] // k.shape[1])
    return causal_softmax_attention(np.einsum("ihd,jhd->hij", q, k[:, src]) * scale, v[:, src])


def rotate_heads(x, rot):
    """Interleaved rotation of [T, heads, d] by each row's place (no spec: as it is)."""
    return rotate_pairs(x, np.arange(len(x)), rot) if rot else x


def normed_attention(h, w, p, m, eps, shared=None):
    """One norm over all query rows and one over all key rows, ahead of the split into heads."""
    T, dim = len(h), m["dim"]
    q = rms_norm(h @ w[p + "q"].T, w[p + "q.norm"], eps).reshape(T, m["heads"], dim)
    k = rms_norm(h @ w[p + "k"].T, w[p + "k.norm"], eps).reshape(T, m["kv_heads"], dim)
    v = (h @ w[p + "v"].T).reshape(T, m["kv_heads"], m["vdim"])
    o = grouped_attention(rotate_heads(q, m.get("rot")), rotate_heads(k, m.get("rot")), v, m["scale"])
    return o.reshape(T, -1) @ w[p + "o"].T


def key_value_attention(h, w, p, m, eps, shared=None):
    """The keys as projected are the values; a logistic gate on the concatenated heads."""
    T = len(h)
    q, k = (h @ w[p + "q"].T).reshape(T, m["heads"], m["dim"]), (h @ w[p + "k"].T).reshape(T, m["kv_heads"], m["dim"])
    o = grouped_attention(rotate_heads(q, m.get("rot")), rotate_heads(k, m.get("rot")), k, m["scale"])
    return (o.reshape(T, -1) * sigmoid(h @ w[p + "g"].T)) @ w[p + "o"].T


def latent_of(h, w, p, m, eps):
    """What a latent layer caches per token: the normed latent and the rotated key part."""
    rank = m["kv_rank"]
    kv = h @ w[p + "dkv"].T
    return rms_norm(kv[:, :rank], w[p + "dkv.norm"], eps), rotate_halves(kv[:, rank:], np.arange(len(h)), m["rot"])


def gated_latent_attention(h, w, p, m, eps, shared=None):
    """Half-split rotation and a logistic gate; `shared`: another layer's latents and rotated key parts."""
    T = len(h)
    H, dim, rd, dv = m["heads"], m["dim"], m["rot_dim"], m["vdim"]
    c, kr = shared if shared is not None else latent_of(h, w, p, m, eps)
    cq = rms_norm(h @ w[p + "dq"].T, w[p + "dq.norm"], eps)
    q = (cq @ w[p + "uq"].T).reshape(T, H, dim + rd)
    qr = rotate_halves(q[..., dim:], np.arange(T), m["rot"])
    kn, v = (c @ w[p + "uk"].T).reshape(T, H, dim), (c @ w[p + "uv"].T).reshape(T, H, dv)
    scores = (np.einsum("ihd,jhd->hij", q[..., :dim], kn) + np.einsum("ihd,jd->hij", qr, kr)) * m["scale"]
    o = causal_softmax_attention(scores, v).reshape(T, H * dv)
    return (o * sigmoid(h @ w[p + "g"].T)) @ w[p + "o"].T


def gated_feed_forward(h, w, p):
    g, u = (h @ w[p + n].T + w[p + n + ".b"] for n in ("gate", "up"))
    return (silu(g) * u) @ w[p + "down"].T + w[p + "down.b"]


def clamped_expert(h, w, p, limit):
    g, u = np.minimum(h @ w[p + "gate"].T, limit), np.clip(h @ w[p + "up"].T, -limit, limit)
    return (g * sigmoid(1.702 * g) * (u + 1.0)) @ w[p + "down"].T


def route(z, r):
    """Router logits [T, E] -> weights [T, E], zero where an expert is not chosen."""
    T, E = z.shape
    s = np.exp(z - z.max(axis=-1, keepdims=True))
    s /= s.sum(axis=-1, keepdims=True)
    out = np.zeros_like(s)
    groups = r.get("groups") or dict(count=1, keep=1)
    size = E // groups["count"]
    for t in range(T):
        best = np.argsort(-s[t].reshape(groups["count"], size).max(axis=-1), kind="stable")[:groups["keep"]]
        open_to = np.where(np.isin(np.arange(E) // size, best), s[t], -1.0)
        chosen = np.argsort(-open_to, kind="stable")[:r["top"]]
        out[t, chosen] = s[t, chosen] / (s[t, chosen].sum() + 1e-20) * r["scale"]
    return out


def mixture(h, w, p, mlp):
    r = mlp["router"]
    weight = route(h @ w[p + "router"].T, r)
    y = np.zeros_like(h)
    for e in range(r["experts"]):
        t = np.nonzero(weight[:, e])[0]
        if len(t):
            y[t] += weight[t, e, None] * clamped_expert(h[t], w, f"{p}e{e}.", mlp["expert"]["limit"])
    return y


SHARED_AHEAD_MIXERS = {"attention": normed_attention, "attention_2": key_value_attention, "latent_attention": gated_latent_attention}


def forward_shared_norm(cfg, w, tokens, want_layers=False):
    """One norm ahead of each layer; the mixer and the feed-forward both read it and join the stream together."""
    eps = cfg["norm"]["eps"]
    x = np.asarray(w["embed"], np.float64)[np.asarray(tokens)] * cfg["embedding"]["scale"]
    states, latents = [], {}
    for i, layer in enumerate(cfg["layers"]):
        p, m, mlp = f"l{i}.", layer["mixer"], layer.get("mlp")
        h = rms_norm(x, w[p + "norm1"], eps)
        shared = None
        if layer["type"] == "latent_attention":
            if m.get("kv_from") is None:
                latents[i] = latent_of(h, w, p + "mix.", m, eps)
            shared = latents[i if m.get("kv_from") is None else m["kv_from"]]
        y = SHARED_AHEAD_MIXERS[layer["type"]](h, w, p + "mix.", m, eps, shared)
        if mlp:
            y = y + (gated_feed_forward(h, w, p + "mlp.") if mlp["kind"] == "dense" else mixture(h, w, p + "mlp.", mlp))
        x = x + y
        states.append(x)
    logits = rms_norm(x, w["final.norm"], eps) @ w["head"].T
    return (logits, np.stack(states)) if want_layers else logits


# ---- Minodra ---------------------------------------------------------------------------------------
def bigram_rows(tokens, buckets, mul_prev, mul_cur):
    """Row of the bigram table per place: a hash of the previous and the own token; the last row at the start."""
    t = [int(x) for x in tokens]
    return np.array([buckets] + [(a * mul_prev + b * mul_cur) % buckets for a, b in zip(t, t[1:])])


def scalar_norm(x, g, eps):
    """Divided by its root mean square, times one number."""
    return divide_by_rms(np.asarray(x, np.float64), eps) * float(np.asarray(g).reshape(()))


def softcap(logits, cap):
    return cap * np.tanh(logits / cap)


def with_recent(h, w):
    """A row plus a causal convolution over it and the rows before it."""
    return h + causal_conv(h, w)


def softmax_with_learned_sink(scores, seen, sink):
    """scores [H, T, T], sink [H] in score units: exp(sink) joins the sum, without key or value."""
    s = np.where(seen, scores, -np.inf)
    m = np.maximum(s.max(axis=-1, keepdims=True), sink[:, None, None])
    p = np.exp(s - m)
    return p / (p.sum(axis=-1, keepdims=True) + np.exp(sink[:, None, None] - m))


def sink_latent_attention(h, w, p, m, eps):
    """No rotation; a learned sink and one logistic output gate per head."""
    T, H, dim, dv = len(h), m["heads"], m["dim"], m["vdim"]
    cq = rms_norm(h @ w[p + "dq"].T, w[p + "dq.norm"], eps)
    c = rms_norm(h @ w[p + "dkv"].T, w[p + "dkv.norm"], eps)
    q, k, v = ((x @ w[p + n].T).reshape(T, H, d) for x, n, d in ((cq, "uq", dim), (c, "uk", dim), (c, "uv", dv)))
    a = softmax_with_learned_sink(np.einsum("ihd,jhd->hij", q, k) * m["scale"], window_mask(T, None), w[p + "sink"])
    o = np.einsum("hij,jhd->ihd", a, v) * sigmoid(h @ w[p + "g"].T)[:, :, None]
    return o.reshape(T, H * dv) @ w[p + "o"].T


def silu_pair_feed_forward(h, w, p):
    return (silu(h @ w[p + "gate"].T) * (h @ w[p + "up"].T)) @ w[p + "down"].T


def corrected_route(z, correction, top):
    """Logistic scores; the largest scores plus correction are chosen, the plain scores are the weights."""
    s = sigmoid(z)
    out = np.zeros_like(s)
    for t in range(len(z)):
        chosen = np.argsort(-(s[t] + correction), kind="stable")[:top]
        out[t, chosen] = s[t, chosen]
    return out


def shared_mixture(h, w, p, mlp):
    """Squared-ReLU experts, the chosen ones weighted; one more for every token behind a logistic gate."""
    weight = corrected_route(h @ w[p + "router"].T, w[p + "correction"], mlp["router"]["top"])
    y = np.zeros_like(h)
    for e in range(mlp["router"]["experts"]):
        t = np.nonzero(weight[:, e])[0]
        if len(t):
            y[t] += weight[t, e, None] * feed_forward(h[t], w, f"{p}e{e}.")
    if mlp.get("shared"):
        y += sigmoid(h @ w[p + "shared.sg"].T) * feed_forward(h, w, p + "shared.")
    return y


def gated_sublayer(x, w, p, n, sublayer, eps):
    """x plus the sublayer's output through a logistic gate; both read the normed stream, the sublayer behind a convolution."""
    h = scalar_norm(x, w[f"{p}norm{n}"], eps)
    return x + sublayer(with_recent(h, w[f"{p}canon{n}"])) * sigmoid(h @ w[f"{p}rg{n}"].T + w[f"{p}rg{n}.b"])


def forward_gated(cfg, w, tokens, want_layers=False):
    eps, b = cfg["norm"]["eps"], cfg["embedding"].get("bigram")
    x = np.asarray(w["embed"], np.float64)[np.asarray(tokens)] * cfg["embedding"]["scale"]
    if b:
        x = x + w["bigram"][bigram_rows(tokens, b["buckets"], b["mul_prev"], b["mul_cur"])]
    x = scalar_norm(x, w["embed.norm"], eps)
    states = []
    for i, layer in enumerate(cfg["layers"]):
        p, mlp = f"l{i}.", layer.get("mlp")
        x = gated_sublayer(x, w, p, 1, lambda h: sink_latent_attention(h, w, p + "mix.", layer["mixer"], eps), eps)
        if mlp:
            ff = silu_pair_feed_forward if mlp["kind"] == "dense" else (lambda h, w, q: shared_mixture(h, w, q, mlp))
            x = gated_sublayer(x, w, p, 2, lambda h: ff(h, w, p + "mlp."), eps)
        states.append(x)
    logits = softcap(scalar_norm(x, w["final.norm"], eps) @ w["head"].T, cfg["logit_softcap"])
    return (logits, np.stack(states)) if want_layers else logits


def forward(cfg, w, tokens, want_layers=False):
    """Logits [T, vocab] of one sequence (and the residual stream after every layer)."""
    if cfg["architecture"] == "Minodra":
        return forward_gated(cfg, w, tokens, want_layers)
    if cfg["architecture"] == "Lofudra":
        return forward_sandwich(cfg, w, tokens, want_layers)
    if cfg["architecture"] == "Fobanex":
        return forward_shared_norm(cfg, w, tokens, want_layers)
    eps = cfg["norm"]["eps"]
    x = np.asarray(w["embed"], np.float64)[np.asarray(tokens)]
    states = []
    for i, layer in enumerate(cfg["layers"]):
        p = f"l{i}."
        x = x + rms_norm(MIXERS[layer["type"]](x, w, p + "mix.", layer["mixer"], eps), w[p + "norm1"], eps)
        if layer.get("mlp"):
            x = x + rms_norm(feed_forward(x, w, p + "mlp."), w[p + "norm2"], eps)
        states.append(x)
    logits = rms_norm(x, w["final.norm"], eps) @ w["head"].T * cfg["logit_scale"]
    cap = cfg["logit_softcap"]
    logits = cap * np.tanh(logits / cap)
    return (logits, np.stack(states)) if want_layers else logits


def greedy(cfg, w, prompt, n):
    """n greedy tokens after `prompt`, and the logits each was chosen from."""
    toks, logits = list(prompt), []
    for _ in range(n):
        lg = forward(cfg, w, toks)[-1]
        logits.append(lg)
        toks.append(int(np.argmax(lg)))
    return toks[len(prompt):], np.stack(logits)
