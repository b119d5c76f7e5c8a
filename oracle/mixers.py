"""Plain float64 restatement of the layers a mixed decoder is made of (gated delta rule, latent attention, sliding-window
attention beside lightning attention, gated feed-forwards), one function per mechanism, token by token where the mechanism
is a recurrence.  Test infrastructure: written from the equations, shares no code with the kernels, and is slow on purpose.

A model is (config, tensors): the configuration dictionary of a Zuselix or Matalix model directory and a dictionary
name -> float array.  Every function works on float64 NumPy arrays.
"""
from __future__ import annotations

import numpy as np


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def silu(z):
    return z * sigmoid(z)


def softplus(z):
    return np.log1p(np.exp(-np.abs(z))) + np.maximum(z, 0.0)


def layer_norm(x, w, eps):
    c = x - x.mean(-1, keepdims=True)
    return c / np.sqrt((c * c).mean(-1, keepdims=True) + eps) * w


def rms_norm(x, w, eps):
    return x / np.sqrt((x * x).mean(-1, keepdims=True) + eps) * w


def unit(x):
    return x / np.sqrt((x * x).sum(-1, keepdims=True) + 1e-6)


def sinusoid(positions, width):
    """row p: entry 2i = sin(p f_i), entry 2i + 1 = cos(p f_i), f_i = 10000^(-2i / width)"""
    p = np.asarray(positions, np.float64)[:, None]
    d = np.arange(width)
    a = p * 10000.0 ** (-(d - d % 2) / width)
    return np.where(d % 2 == 0, np.sin(a), np.cos(a))


def short_conv(x, taps):
    """causal convolution per channel over (tokens, channels), then silu; taps[c, -1] meets the token itself"""
    n = taps.shape[1]
    out = np.zeros_like(x)
    for t in range(x.shape[0]):
        for j in range(n):
            if t - j >= 0:
                out[t] += taps[:, n - 1 - j] * x[t - j]
    return silu(out)


def delta_recurrence(q, k, v, g, beta):
    """one head: q, k (tokens, dim), v (tokens, vdim), g and beta (tokens); returns (o, final state)"""
    S = np.zeros((k.shape[1], v.shape[1]))
    o = np.zeros_like(v)
    for t in range(len(g)):
        S = g[t] * S
        u = beta[t] * (v[t] - S.T @ k[t])
        S = S + np.outer(k[t], u)
        o[t] = S.T @ q[t]
    return o, S


def delta_mixer(h, m, w, eps):
    """h (tokens, width); m: the mixer's sizes; w(name): its tensors"""
    T, H, KH, dk, dv = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = unit(short_conv(h @ w("q").T, w("q.conv")).reshape(T, KH, dk)) * dk ** -0.5
    k = unit(short_conv(h @ w("k").T, w("k.conv")).reshape(T, KH, dk))
    v = short_conv(h @ w("v").T, w("v.conv")).reshape(T, H, dv)
    beta = sigmoid(h @ w("b").T)
    g = np.exp(-np.exp(w("A_log")) * softplus(h @ w("a").T + w("dt_bias")))
    gate = silu(h @ w("g").T).reshape(T, H, dv)
    o = np.zeros((T, H, dv))
    for n in range(H):
        kh = n // (H // KH)
        o[:, n], _ = delta_recurrence(q[:, kh], k[:, kh], v[:, n], g[:, n], beta[:, n])
    return (rms_norm(o, w("norm"), eps) * gate).reshape(T, -1) @ w("o").T


def sink_softmax(s, sink):
    """exp(s_j) / (exp(sink) + sum_j exp(s_j)) over the last axis; -inf entries do not take part"""
    top = np.maximum(s.max(-1), sink)
    e = np.exp(s - top[..., None])
    return e / (np.exp(sink - top) + e.sum(-1))[..., None]


def latent_attention_mixer(h, m, w, eps):
    T, H, dk, dv = h.shape[0], m["heads"], m["dim"], m["vdim"]
    q = (h @ w("q").T).reshape(T, H, dk)
    c = rms_norm(h @ w("dkv").T, w("dkv.norm"), eps)
    k = (c @ w("uk").T).reshape(T, H, dk)
    v = (c @ w("uv").T).reshape(T, H, dv)
    gate = sigmoid(h @ w("g").T)
    o = np.zeros((T, H, dv))
    hidden = np.triu(np.full((T, T), -np.inf), 1)
    for n in range(H):
        o[:, n] = sink_softmax(q[:, n] @ k[:, n].T * m["scale"] + hidden, w("sink")[n]) @ v[:, n]
    return (o.reshape(T, -1) * gate) @ w("o").T


def dense_mlp(h, w):
    return (silu(h @ w("gate").T) * (h @ w("up").T)) @ w("down").T


MIXERS = {"delta": delta_mixer, "latent_attention": latent_attention_mixer}


def zuselix(config, tensors, tokens):
    """-> (logits (tokens, vocab), residual stream after every layer (layers, tokens, width))"""
    t = {k: np.asarray(v, np.float64) for k, v in tensors.items()}
    eps = config["norm"]["eps"]
    x = t["embed"][np.asarray(tokens)] + sinusoid(range(len(tokens)), config["width"])
    stream = []
    for i, layer in enumerate(config["layers"]):
        p = f"l{i}."
        mixer = MIXERS[layer["type"]]
        x = x + mixer(layer_norm(x, t[p + "norm1"], eps), layer["mixer"], lambda n: t[p + "mix." + n], eps)
        if layer["mlp"] is not None:
            x = x + dense_mlp(layer_norm(x, t[p + "norm2"], eps), lambda n: t[p + "mlp." + n])
        stream.append(x)
    logits = layer_norm(x, t["final.norm"], eps) @ t["head"].T
    cap = config["logit_softcap"]
    return cap * np.tanh(logits / cap) if cap else logits, np.array(stream)


# ---- Matalix ----
def yarn(rot):
    """rotation frequencies (dims / 2) and the factor of cosine and sine: slow rotations are stretched by `factor`, fast
    ones are left, a linear ramp over the pair index lies between"""
    dims, base, sc = rot["dims"], rot["base"], rot.get("scaling")
    if sc is None:
        return base ** (-2.0 * np.arange(dims // 2) / dims), 1.0

    def pair_that_turns(times):  # the (real-valued) pair that turns `times` times over the original context
        return dims * np.log(sc["original"] / (2 * np.pi * times)) / (2 * np.log(base))
    lo = max(np.floor(pair_that_turns(sc["fast"])), 0)
    hi = min(np.ceil(pair_that_turns(sc["slow"])), dims - 1)
    i = np.arange(dims // 2)
    f = base ** (-2.0 * i / dims)
    ramp = np.clip((i - lo) / max(hi - lo, 0.001), 0.0, 1.0)
    return f / sc["factor"] * ramp + f * (1.0 - ramp), 0.1 * np.log(sc["factor"]) + 1.0


def rotate_half(x, positions, freqs, mscale):
    """x (tokens, heads, dim): entries i and i + n of a head are a pair (n = len(freqs)), entries from 2 n on stay"""
    n = len(freqs)
    a = np.asarray(positions, np.float64)[:, None, None] * freqs
    c, s = np.cos(a) * mscale, np.sin(a) * mscale
    u, v = x[..., :n], x[..., n:2 * n]
    return np.concatenate([u * c - v * s, v * c + u * s, x[..., 2 * n:]], -1)


def window_attention(h, m, w, eps, bias=True, qk_norm=True, sink=0.0, gate=True):
    """grouped-query attention over the last mask.size positions; sink: a score per head or for all of them (-inf = none)"""
    T, H, G, dk, dv = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k, v = (h @ w(n).T + (w(n + ".b") if bias else 0.0) for n in ("q", "k", "v"))
    if qk_norm:
        q, k = rms_norm(q, w("q.norm"), eps), rms_norm(k, w("k.norm"), eps)
    q, k, v = q.reshape(T, H, dk), k.reshape(T, G, dk), v.reshape(T, G, dv)
    if m["rot"] is not None:
        freqs, mscale = yarn(m["rot"])
        q, k = rotate_half(q, range(T), freqs, mscale), rotate_half(k, range(T), freqs, mscale)
    back = np.arange(T)[:, None] - np.arange(T)[None, :]
    hidden = np.where((back >= 0) & (back < m["mask"]["size"]), 0.0, -np.inf)
    sink = np.broadcast_to(sink, (H,))
    o = np.zeros((T, H, dv))
    for n in range(H):
        g = n // (H // G)
        o[:, n] = sink_softmax(q[:, n] @ k[:, g].T * m["scale"] + hidden, sink[n]) @ v[:, g]
    return (o.reshape(T, -1) * (sigmoid(h @ w("g").T) if gate else 1.0)) @ w("o").T


def lightning_recurrence(q, k, v, decay):
    """one head: q, k (tokens, dim), v (tokens, vdim); returns (o, final state)"""
    S = np.zeros((k.shape[1], v.shape[1]))
    o = np.zeros_like(v)
    for t in range(len(q)):
        S = decay * S + np.outer(k[t], v[t])
        o[t] = S.T @ q[t]
    return o, S


def lightning_attention(h, m, w, eps):
    T, H, dk, dv = h.shape[0], m["heads"], m["dim"], m["vdim"]
    q, k = silu(h @ w("q").T).reshape(T, H, dk), silu(h @ w("k").T).reshape(T, H, dk)
    v = silu(h @ w("v").T).reshape(T, H, dv)
    o = np.zeros((T, H, dv))
    for n in range(H):
        o[:, n], _ = lightning_recurrence(q[:, n], k[:, n], v[:, n], m["decay"][n])
    return (rms_norm(o.reshape(T, -1), w("norm"), eps) * sigmoid(h @ w("g").T)) @ w("o").T


def parallel_mixer(h, m, w, eps):
    return (m["left_scale"] * window_attention(h, m["left"], lambda n: w("left." + n), eps)
            + m["right_scale"] * lightning_attention(h, m["right"], lambda n: w("right." + n), eps))


def clamped_mlp(h, limit, w):
    g = np.minimum(h @ w("gate").T, limit)
    u = np.clip(h @ w("up").T, -limit, limit)
    return (g * sigmoid(1.702 * g) * (u + 1.0)) @ w("down").T


def matalix(config, tensors, tokens):
    """-> (logits (tokens, vocab), residual stream after every layer run (layer runs, tokens, width))"""
    t = {k: np.asarray(v, np.float64) for k, v in tensors.items()}
    eps, loop = config["norm"]["eps"], config.get("loop") or {"start": 0, "stop": 0, "times": 1}
    x0 = x = t["embed"][np.asarray(tokens)]
    stream = []

    def run(i, x):
        layer, p = config["layers"][i], f"l{i}."
        x = x + t[p + "ls1"] * parallel_mixer(rms_norm(x, 1.0 + t[p + "norm1"], eps), layer["mixer"], lambda n: t[p + "mix." + n], eps)
        if layer["mlp"] is not None:
            x = x + t[p + "ls2"] * clamped_mlp(rms_norm(x, 1.0 + t[p + "norm2"], eps), layer["mlp"]["limit"], lambda n: t[p + "mlp." + n])
        stream.append(x)
        return x
    for i in range(loop["start"]):
        x = run(i, x)
    for p in range(loop["times"]):
        if p:
            x = x + x0
        for i in range(loop["start"], loop["stop"]):
            x = run(i, x)
    for i in range(loop["stop"], len(config["layers"])):
        x = run(i, x)
    return rms_norm(x, 1.0 + t["final.norm"], eps) @ t["embed"].T, np.array(stream)
