"""Small random Zuselix and Matalix models for the tests: a configuration as a model directory's config.json holds it, and tensors
whose values bf16 holds exactly."""
import numpy as np

from caten_amd import llm, synth
from caten_amd.quant import from_bf16, to_bf16


def delta(heads=4, kv_heads=2, dim=16, vdim=32, conv=4, ff=None):
    return {"type": "delta", "mixer": dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, conv=conv), "mlp": mlp(ff)}


def latent(heads=4, dim=32, vdim=32, kv_rank=48, scale=0.2, ff=None):
    return {"type": "latent_attention", "mixer": dict(heads=heads, dim=dim, vdim=vdim, kv_rank=kv_rank, scale=scale), "mlp": mlp(ff)}


def mlp(ff):
    return None if ff is None else {"kind": "dense", "ff": ff}


def config(layers, width=128, vocab=320, eps=1e-5, cap=20.0):
    return {"architecture": "Zuselix", "layers": layers, "logit_softcap": cap, "norm": {"eps": eps}, "vocab": vocab, "width": width}


def window(heads=4, kv_heads=2, dim=32, vdim=32, size=24, scale=0.2, dims=None, base=10000.0, factor=8.0, original=64, fast=8.0, slow=1.0):
    return dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, scale=scale, mask={"size": size},
                rot=dict(base=base, dims=dim if dims is None else dims, scaling=dict(factor=factor, original=original, fast=fast, slow=slow)))


def lightning(heads=3, dim=16, vdim=32, decay=None):
    return dict(heads=heads, dim=dim, vdim=vdim, decay=[1.0 - 0.4 * 0.3 ** h for h in range(heads)] if decay is None else decay)


def parallel(left=None, right=None, left_scale=0.7, right_scale=1.2, ff=None, limit=3.0):
    return {"type": "parallel", "mixer": dict(left=left or window(), left_scale=left_scale, right=right or lightning(), right_scale=right_scale),
            "mlp": None if ff is None else {"kind": "dense", "ff": ff, "limit": limit}}


def matalix(layers, width=128, vocab=320, eps=1e-5, loop=None):
    return {"architecture": "Matalix", "layers": layers, "loop": loop or dict(start=0, stop=1, times=1), "norm": {"eps": eps}, "vocab": vocab, "width": width}


def as_bf16(a):
    """the nearest values that bf16 holds"""
    a = np.asarray(a, np.float32)
    return from_bf16(to_bf16(a.ravel())).reshape(a.shape)


def weights(cfg, seed=0, **scale):
    """name -> fp32 array of bf16 values; scale: factor per tensor-name suffix"""
    rng = np.random.default_rng(seed)
    shapes, tensor = (synth.matalix_shapes, synth.matalix_tensor) if cfg["architecture"] == "Matalix" else (synth.zuselix_shapes, synth.zuselix_tensor)
    out = {}
    for name, shape in shapes(cfg).items():
        a = tensor(name, shape, rng)
        for suffix, f in scale.items():
            if name.endswith("." + suffix):
                a = a * f
        out[name] = as_bf16(a)
    return out


def raw_tensors(w):
    """as safetensors.read returns them"""
    return {k: ("bf16", a.shape, to_bf16(a.ravel()).view(np.uint8)) for k, a in w.items()}


def session(cfg, w, dtype="float32", max_seq=256, **over):
    """an open session; dtype as llm.load_model takes it"""
    c = dict(llm.ARCHITECTURES[cfg["architecture"]][0](cfg), max_seq=max_seq, **over)
    if dtype == "float32":
        c["precision"] = 0
    sd = llm.safetensors_state_dict(raw_tensors(w), widen=dtype == "float32")
    return llm.MixedTransformer(c).load_state_dict(sd)


def tokens(cfg, n, seed=0):
    return [int(t) for t in np.random.default_rng(1000 + seed).integers(0, cfg["vocab"], n)]
