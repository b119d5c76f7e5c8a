"""Plain float64 restatement of the layers a mixed decoder is made of (gated delta rule, latent attention, gated
feed-forward), one function per mechanism, token by token where the mechanism is a recurrence.  Test infrastructure:
written from the equations, shares no code with the kernels, and is slow on purpose.

A model is (config, tensors): the configuration dictionary of a Zuselix model directory and a dictionary
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
