"""Plain, slow statement of the layer-stack models (per-layer mixers: latent attention and the
channel-decay delta rule) in numpy double precision.

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


MIXERS = {"latent_attention": latent_attention, "channel_delta": channel_delta}


def feed_forward(x, w, p):
    return squared_relu(x @ w[p + "up"].T) @ w[p + "down"].T


def forward(cfg, w, tokens, want_layers=False):
    """Logits [T, vocab] of one sequence (and the residual stream after every layer)."""
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
