"""Small random Zuselix models for the tests: a configuration as a model directory's config.json holds it, and tensors
whose values bf16 holds exactly."""
import numpy as np

from caten_amd import llm
from caten_amd.quant import from_bf16, to_bf16


def delta(heads=4, kv_heads=2, dim=16, vdim=32, conv=4, ff=None):
    return {"type": "delta", "mixer": dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, conv=conv), "mlp": mlp(ff)}


def latent(heads=4, dim=32, vdim=32, kv_rank=48, scale=0.2, ff=None):
    return {"type": "latent_attention", "mixer": dict(heads=heads, dim=dim, vdim=vdim, kv_rank=kv_rank, scale=scale), "mlp": mlp(ff)}


def mlp(ff):
    return None if ff is None else {"kind": "dense", "ff": ff}


def config(layers, width=128, vocab=320, eps=1e-5, cap=20.0):
    return {"architecture": "Zuselix", "layers": layers, "logit_softcap": cap, "norm": {"eps": eps}, "vocab": vocab, "width": width}


def shapes(cfg):
    W, V = cfg["width"], cfg["vocab"]
    out = {"embed": (V, W), "final.norm": (W,), "head": (V, W)}
    for i, l in enumerate(cfg["layers"]):
        m, p = l["mixer"], f"l{i}."
        out[p + "norm1"] = (W,)
        H, dk, dv = m["heads"], m["dim"], m["vdim"]
        if l["type"] == "delta":
            K, n = m["kv_heads"] * dk, m["conv"]
            out.update({p + "mix.q": (K, W), p + "mix.q.conv": (K, n), p + "mix.k": (K, W), p + "mix.k.conv": (K, n),
                        p + "mix.v": (H * dv, W), p + "mix.v.conv": (H * dv, n), p + "mix.b": (H, W), p + "mix.a": (H, W),
                        p + "mix.A_log": (H,), p + "mix.dt_bias": (H,), p + "mix.norm": (dv,), p + "mix.g": (H * dv, W),
                        p + "mix.o": (W, H * dv)})
        else:
            r = m["kv_rank"]
            out.update({p + "mix.q": (H * dk, W), p + "mix.dkv": (r, W), p + "mix.dkv.norm": (r,), p + "mix.uk": (H * dk, r),
                        p + "mix.uv": (H * dv, r), p + "mix.sink": (H,), p + "mix.g": (H * dv, W), p + "mix.o": (W, H * dv)})
        if l["mlp"] is not None:
            F = l["mlp"]["ff"]
            out.update({p + "norm2": (W,), p + "mlp.gate": (F, W), p + "mlp.up": (F, W), p + "mlp.down": (W, F)})
    return out


def weights(cfg, seed=0, **scale):
    """name -> fp32 array of bf16 values; scale: factor per tensor-name suffix"""
    rng = np.random.default_rng(seed)
    out = {}
    for name, shape in shapes(cfg).items():
        a = rng.standard_normal(shape)
        last = name.rsplit(".", 1)[-1]
        if "norm" in last:
            a = 1.0 + 0.2 * a
        elif last == "A_log":
            a = np.log(rng.uniform(0.05, 2.0, shape))
        elif last == "dt_bias":
            a = a - 2.0
        elif last == "sink":
            a = 1.5 * a
        elif last == "conv":
            a = a * 0.6
        elif name != "embed":
            a = a / np.sqrt(shape[-1])
        for suffix, f in scale.items():
            if name.endswith("." + suffix):
                a = a * f
        out[name] = from_bf16(to_bf16(a.astype(np.float32).ravel())).reshape(shape)
    return out


def raw_tensors(w):
    """as safetensors.read returns them"""
    return {k: ("bf16", a.shape, to_bf16(a.ravel()).view(np.uint8)) for k, a in w.items()}


def session(cfg, w, dtype="float32", max_seq=256, **over):
    """an open session; dtype as llm.load_model takes it"""
    c = dict(llm.zuselix_config(cfg), max_seq=max_seq, **over)
    if dtype == "float32":
        c["precision"] = 0
    sd = llm.safetensors_state_dict(raw_tensors(w), widen=dtype == "float32")
    return llm.MixedTransformer(c).load_state_dict(sd)


def tokens(cfg, n, seed=0):
    return [int(t) for t in np.random.default_rng(1000 + seed).integers(0, cfg["vocab"], n)]
