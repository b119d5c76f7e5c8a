"""Synthetic, seeded weights and prompts of the shapes the decode path is measured on.

Caten's own RNG (threefry2x32 built from graph ops, source/api/initializers.lisp:55-99)
has no golden stream, so inputs are generated here with NumPy ``default_rng(seed)``
and fed to both the HIP path and the CPU oracle.
"""
from __future__ import annotations

import numpy as np

# apps/gpt2/gpt2.lisp:36-44 parameter table (+ the tiny shapes the tests use)
GPT2_CONFIGS = {
    "gpt2": dict(n_layers=12, n_heads=12, dim=768, ffn=3072, vocab=50257, max_seq=1024, eps=1e-5),
    "gpt2-medium": dict(n_layers=24, n_heads=16, dim=1024, ffn=4096, vocab=50257, max_seq=1024, eps=1e-5),
    "gpt2-large": dict(n_layers=36, n_heads=20, dim=1280, ffn=5120, vocab=50257, max_seq=1024, eps=1e-5),
    "gpt2-xl": dict(n_layers=48, n_heads=25, dim=1600, ffn=6400, vocab=50257, max_seq=1024, eps=1e-5),
    "gpt2-tiny": dict(n_layers=2, n_heads=4, dim=256, ffn=1024, vocab=1000, max_seq=64, eps=1e-5),
    "gpt2-mini": dict(n_layers=3, n_heads=12, dim=768, ffn=3072, vocab=5003, max_seq=128, eps=1e-5),
}

LLAMA_CONFIGS = {
    "llama-1.1b": dict(n_layers=22, n_heads=32, n_kv_heads=4, dim=2048, ffn=5632, vocab=32000,
                       max_seq=2048, eps=1e-5, rope_base=10000.0),
    "llama-tiny": dict(n_layers=2, n_heads=8, n_kv_heads=2, dim=512, ffn=1024, vocab=1000,
                       max_seq=64, eps=1e-5, rope_base=10000.0),
}


def gpt2_weights(cfg: dict, seed: int = 0) -> dict:
    """Random-init fp32 weights ~N(0,0.02); LayerNorm gamma~N(1,0.02), beta~N(0,0.02)."""
    rng = np.random.default_rng(seed)
    D, F, V, L = cfg["dim"], cfg["ffn"], cfg["vocab"], cfg["n_layers"]

    def n(*shape, mean=0.0):
        return (mean + 0.02 * rng.standard_normal(shape, dtype=np.float32)).astype(np.float32)

    w = dict(wte=n(V, D), wpe=n(cfg["max_seq"], D), lnf_g=n(D, mean=1.0), lnf_b=n(D), lm_head=n(V, D))
    for k in ("ln1_g", "ln1_b", "attn_w", "attn_b", "proj_w", "proj_b",
              "ln2_g", "ln2_b", "fc_w", "fc_b", "fc2_w", "fc2_b"):
        w[k] = []
    for _ in range(L):
        w["ln1_g"].append(n(D, mean=1.0)); w["ln1_b"].append(n(D))
        w["attn_w"].append(n(3 * D, D)); w["attn_b"].append(n(3 * D))
        w["proj_w"].append(n(D, D)); w["proj_b"].append(n(D))
        w["ln2_g"].append(n(D, mean=1.0)); w["ln2_b"].append(n(D))
        w["fc_w"].append(n(F, D)); w["fc_b"].append(n(F))
        w["fc2_w"].append(n(D, F)); w["fc2_b"].append(n(D))
    return w


GPT2_LINEAR_KEYS = ("attn_w", "proj_w", "fc_w", "fc2_w")  # + "lm_head"
LLAMA_LINEAR_KEYS = ("wq", "wk", "wv", "wo", "w_gate", "w_up", "w_down")  # + "lm_head"


def llama_weights(cfg: dict, seed: int = 0, threads: int = 1) -> dict:
    """Random-init fp32 weights ~N(0,0.02), norm weights ~N(1,0.02).  `threads` > 1 draws every tensor from a
    generator of its own (seeded by (seed, tensor number)) on a thread pool: other values than the serial stream
    gives, the same distribution, and a 1.1 B-parameter model in seconds instead of a minute."""
    D, F, V, L = cfg["dim"], cfg["ffn"], cfg["vocab"], cfg["n_layers"]
    KD = D // cfg["n_heads"] * cfg["n_kv_heads"]
    if threads > 1:
        from concurrent.futures import ThreadPoolExecutor
        per_layer = {"attn_norm": ((D,), 1.0), "ffn_norm": ((D,), 1.0), "wq": ((D, D), 0.0), "wk": ((KD, D), 0.0),
                     "wv": ((KD, D), 0.0), "wo": ((D, D), 0.0), "w_gate": ((F, D), 0.0), "w_up": ((F, D), 0.0),
                     "w_down": ((D, F), 0.0)}
        jobs = [("tok_emb", None, (V, D), 0.0), ("norm_w", None, (D,), 1.0), ("lm_head", None, (V, D), 0.0)]
        jobs += [(k, l, sh, mean) for l in range(L) for k, (sh, mean) in per_layer.items()]

        def draw(i):
            _, _, shape, mean = jobs[i]
            a = np.random.default_rng([seed, i]).standard_normal(shape, dtype=np.float32)
            a *= np.float32(0.02)
            if mean:
                a += np.float32(mean)
            return a
        with ThreadPoolExecutor(threads) as pool:
            arrs = list(pool.map(draw, range(len(jobs))))
        w = {k: [None] * L for k in per_layer}
        for (k, l, _, _), a in zip(jobs, arrs):
            if l is None:
                w[k] = a
            else:
                w[k][l] = a
        return w
    rng = np.random.default_rng(seed)

    def n(*shape, mean=0.0):
        return (mean + 0.02 * rng.standard_normal(shape, dtype=np.float32)).astype(np.float32)

    w = dict(tok_emb=n(V, D), norm_w=n(D, mean=1.0), lm_head=n(V, D))
    for k in ("attn_norm", "ffn_norm") + LLAMA_LINEAR_KEYS:
        w[k] = []
    for _ in range(L):
        w["attn_norm"].append(n(D, mean=1.0)); w["ffn_norm"].append(n(D, mean=1.0))
        w["wq"].append(n(D, D)); w["wk"].append(n(KD, D)); w["wv"].append(n(KD, D)); w["wo"].append(n(D, D))
        w["w_gate"].append(n(F, D)); w["w_up"].append(n(F, D)); w["w_down"].append(n(D, F))
    return w


def _zuselix(width, ff, heads, kv_heads, rank, blocks, vocab=32000):
    """blocks of two delta layers and a latent-attention layer, each with a feed-forward; heads of 128"""
    delta = {"type": "delta", "mixer": dict(heads=heads, kv_heads=kv_heads, dim=128, vdim=128, conv=4), "mlp": {"kind": "dense", "ff": ff}}
    latent = {"type": "latent_attention", "mixer": dict(heads=heads, dim=128, vdim=128, kv_rank=rank, scale=128 ** -0.5),
              "mlp": {"kind": "dense", "ff": ff}}
    return {"architecture": "Zuselix", "layers": [delta, delta, latent] * blocks, "logit_softcap": 30.0, "norm": {"eps": 1e-5},
            "vocab": vocab, "width": width}


# config.json-shaped configurations beside Llama shapes of the same width, feed-forward, depth and vocabulary
ZUSELIX_CONFIGS = {
    "zuselix-1b": _zuselix(2048, 5632, 16, 8, 512, 7),
    "zuselix-7b": _zuselix(4096, 11008, 32, 16, 512, 5),  # (15 of a 7B model's 32 layers)
}


def zuselix_shapes(config: dict) -> dict:
    """tensor name -> shape of a Zuselix model (cthip_decoder_create_mixed's state-dict keys)"""
    W, V = config["width"], config["vocab"]
    out = {"embed": (V, W), "final.norm": (W,), "head": (V, W)}
    for i, layer in enumerate(config["layers"]):
        m, p = layer["mixer"], f"l{i}."
        H, dk, dv = m["heads"], m["dim"], m["vdim"]
        out.update({p + "norm1": (W,), p + "mix.q": (m.get("kv_heads", H) * dk, W), p + "mix.g": (H * dv, W), p + "mix.o": (W, H * dv)})
        if layer["type"] == "delta":
            K, taps = m["kv_heads"] * dk, m["conv"]
            out.update({p + "mix.k": (K, W), p + "mix.v": (H * dv, W), p + "mix.q.conv": (K, taps), p + "mix.k.conv": (K, taps),
                        p + "mix.v.conv": (H * dv, taps), p + "mix.b": (H, W), p + "mix.a": (H, W), p + "mix.A_log": (H,),
                        p + "mix.dt_bias": (H,), p + "mix.norm": (dv,)})
        else:
            r = m["kv_rank"]
            out.update({p + "mix.dkv": (r, W), p + "mix.dkv.norm": (r,), p + "mix.uk": (H * dk, r), p + "mix.uv": (H * dv, r),
                        p + "mix.sink": (H,)})
        if layer["mlp"] is not None:
            F = layer["mlp"]["ff"]
            out.update({p + "norm2": (W,), p + "mlp.gate": (F, W), p + "mlp.up": (F, W), p + "mlp.down": (W, F)})
    return out


def zuselix_tensor(name: str, shape: tuple, rng) -> np.ndarray:
    """one tensor's random fp32 values: unit-variance sums, norm weights around 1, decays and steps of a few tokens to hundreds"""
    last = name.rsplit(".", 1)[-1]
    if last == "A_log":
        return np.log(rng.uniform(0.05, 2.0, shape)).astype(np.float32)
    a = rng.standard_normal(shape, dtype=np.float32)
    if "norm" in last:
        return 1.0 + 0.2 * a
    if last == "dt_bias":
        return a - 2.0
    if last == "sink":
        return 1.5 * a
    if last == "conv":
        return 0.6 * a
    return a if name == "embed" else a / np.float32(np.sqrt(shape[-1]))


def _matalix(width, ff, heads, kv_heads, window, layers, loop, vocab=32000):
    """heads of 128; as many lightning heads of 128 as half the query heads, decays of tens to thousands of tokens"""
    n = heads // 2
    left = dict(heads=heads, kv_heads=kv_heads, dim=128, vdim=128, scale=128 ** -0.5, mask={"size": window},
                rot=dict(base=10000.0, dims=128, scaling=dict(factor=4.0, original=2048, fast=32.0, slow=1.0)))
    right = dict(heads=n, dim=128, vdim=128, decay=[1.0 - 2.0 ** -(4.0 + 6.0 * h / max(n - 1, 1)) for h in range(n)])
    layer = {"type": "parallel", "mixer": dict(left=left, left_scale=0.7, right=right, right_scale=0.6), "mlp": {"kind": "dense", "ff": ff, "limit": 7.0}}
    return {"architecture": "Matalix", "layers": [layer] * layers, "loop": loop, "norm": {"eps": 1e-5}, "vocab": vocab, "width": width}


# config.json-shaped configurations beside Llama shapes of the same width, feed-forward, layer runs, heads and vocabulary
MATALIX_CONFIGS = {
    "matalix-1b": _matalix(2048, 5632, 16, 4, 1024, 16, dict(start=5, stop=11, times=2)),  # (22 layer runs)
    "matalix-7b": _matalix(4096, 11008, 32, 8, 2048, 12, dict(start=4, stop=8, times=2)),  # (16 layer runs)
}


def matalix_shapes(config: dict) -> dict:
    """tensor name -> shape of a Matalix model (cthip_decoder_create_mixed's state-dict keys)"""
    W, V = config["width"], config["vocab"]
    out = {"embed": (V, W), "final.norm": (W,)}
    for i, layer in enumerate(config["layers"]):
        p, a, b = f"l{i}.", layer["mixer"]["left"], layer["mixer"]["right"]
        q, k, v, o = a["heads"] * a["dim"], a["kv_heads"] * a["dim"], a["kv_heads"] * a["vdim"], a["heads"] * a["vdim"]
        qk, ro = b["heads"] * b["dim"], b["heads"] * b["vdim"]
        out.update({p + "norm1": (W,), p + "ls1": (W,)})
        out.update({p + "mix.left." + n: s for n, s in {
            "q": (q, W), "q.b": (q,), "q.norm": (q,), "k": (k, W), "k.b": (k,), "k.norm": (k,), "v": (v, W), "v.b": (v,), "g": (o, W), "o": (W, o)}.items()})
        out.update({p + "mix.right." + n: s for n, s in {
            "q": (qk, W), "k": (qk, W), "v": (ro, W), "g": (ro, W), "norm": (ro,), "o": (W, ro)}.items()})
        if layer["mlp"] is not None:
            F = layer["mlp"]["ff"]
            out.update({p + "norm2": (W,), p + "ls2": (W,), p + "mlp.gate": (F, W), p + "mlp.up": (F, W), p + "mlp.down": (W, F)})
    return out


def matalix_tensor(name: str, shape: tuple, rng) -> np.ndarray:
    """one tensor's random fp32 values: unit-variance sums, norms stored around zero or one as the design has them, layer
    scales around a half, biases that show"""
    last = name.rsplit(".", 1)[-1]
    a = rng.standard_normal(shape, dtype=np.float32)
    if last in ("norm1", "norm2") or name == "final.norm":
        return 0.2 * a
    if last == "norm":
        return 1.0 + 0.2 * a
    if last in ("ls1", "ls2"):
        return 0.5 + 0.15 * a
    if last == "b":
        return 0.3 * a
    return a if name == "embed" else a / np.float32(np.sqrt(shape[-1]))


def prompt(vocab: int, length: int = 16, seed: int = 0) -> list:
    rng = np.random.default_rng(seed + 1000)
    return [int(t) for t in rng.integers(0, vocab, size=length)]
