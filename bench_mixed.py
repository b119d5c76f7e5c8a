#!/usr/bin/env python3
"""Zuselix shapes (gated delta rule and latent attention layers) and Matalix shapes (sliding-window attention beside lightning
attention, some layers run twice) beside Llama shapes of the same width, feed-forward, layer runs, heads and vocabulary, all
with bf16 weights, on one MI355X: greedy decode at short and long contexts and prompts as one batch.
`python bench.py --mixed`, or this file by itself.

Weights are synthetic; one layer of each kind is drawn and loaded into every layer of that kind, each with its own copy in
HBM.  A session's figures are reported only after its logits for a prompt in one forward agree with the same prompt token
by token.  One JSON line per session:
  decode   us per step, the step's algorithmic bytes (cthip_decoder_step_bytes) and their share of 8 TB/s, HIP events
  prefill  ms of a forward (synchronous, host clock), the Linear layers' TFLOP/s
"""
from __future__ import annotations

import argparse
import ctypes as C
import json
import sys
import time

import numpy as np

HBM_PEAK_GBS = 8000.0


def designs() -> dict:
    """name -> (sizes, tensor shapes, random tensor, configuration of a session)"""
    from caten_amd import llm, synth
    return {"zuselix": (synth.ZUSELIX_CONFIGS, synth.zuselix_shapes, synth.zuselix_tensor, llm.zuselix_config),
            "matalix": (synth.MATALIX_CONFIGS, synth.matalix_shapes, synth.matalix_tensor, llm.matalix_config)}


def sizes() -> list:
    return [n for d in designs().values() for n in d[0]]


def design_of(name: str) -> str:
    return next(k for k, d in designs().items() if name in d[0])


def layer_runs(config: dict) -> list:
    """how often each layer runs per token"""
    loop = config.get("loop") or {"start": 0, "stop": 0, "times": 1}
    return [loop["times"] if loop["start"] <= i < loop["stop"] else 1 for i in range(len(config["layers"]))]


def mixed_session(name: str, max_seq: int):
    """(session, cfg, GFLOP of the Linear layers per token, head left out)"""
    from caten_amd import llm
    from caten_amd.quant import to_bf16
    configs, shapes, tensor, to_cfg = designs()[design_of(name)]
    config = configs[name]
    rng, runs = np.random.default_rng(0), layer_runs(config)
    drawn, sd, flop = {}, {}, 0.0
    for key, shape in shapes(config).items():
        layer, _, rest = key.partition(".")
        in_layer = layer[1:].isdigit()
        kind = config["layers"][int(layer[1:])]["type"] + "." + rest if in_layer else key
        if kind not in drawn:
            bits = to_bf16(tensor(key, shape, rng).ravel())
            rows, cols = shape if len(shape) == 2 else (1, shape[0])
            drawn[kind] = llm.Tensor("bf16", bits.view(np.uint8), rows, cols)
        sd[key] = drawn[kind]
        if in_layer and len(shape) == 2 and shape[1] >= 16:
            flop += 2.0 * shape[0] * shape[1] * runs[int(layer[1:])]
    cfg = dict(to_cfg(config), max_seq=max_seq)
    return llm.MixedTransformer(cfg).load_state_dict(sd), cfg, flop / 1e9


def llama_session(name: str, max_seq: int):
    """the Llama shape of the same width, feed-forward, layer runs, heads and vocabulary"""
    from caten_amd import llm, synth
    z = designs()[design_of(name)][0][name]
    m = z["layers"][0]["mixer"]
    m = m.get("left", m)
    cfg = dict(n_layers=sum(layer_runs(z)), dim=z["width"], n_heads=m["heads"], n_kv_heads=m["kv_heads"], ffn=z["layers"][0]["mlp"]["ff"],
               vocab=z["vocab"], max_seq=max_seq, eps=1e-5, rope_base=10000.0)
    one = llm.llama_state_dict(synth.llama_weights(dict(cfg, n_layers=1), seed=0, threads=8), "bf16", threads=8)
    sd = {}
    for key, t in one.items():
        for l in range(cfg["n_layers"]) if key.startswith("layers.0.") else [None]:
            sd[key if l is None else f"layers.{l}." + key[len("layers.0."):]] = t
    D, F, KD = cfg["dim"], cfg["ffn"], cfg["dim"] // cfg["n_heads"] * cfg["n_kv_heads"]
    flop = 2.0 * cfg["n_layers"] * (D * (D + 2 * KD) + D * D + 3 * D * F)
    return llm.make_llama(cfg, sd), cfg, flop / 1e9


def agree(model, vocab: int) -> float:
    """relative error of the last logits: a prompt in one forward against the same prompt token by token"""
    from caten_amd import synth
    toks = synth.prompt(vocab, 40, seed=2)
    _, a = model.forward(toks, len(toks), 0, return_logits=True)
    for i, t in enumerate(toks):
        _, b = model.forward([t], 1, i, return_logits=True)
    return float(np.linalg.norm(a - b) / np.linalg.norm(b))


def decode_us(model, lib, vocab: int, plen: int, steps: int):
    from caten_amd import _lib, synth
    prompt = synth.prompt(vocab, plen, seed=1)
    best = None
    for _ in range(4):
        model.forward(prompt, plen, 0)
        model.generate_on_device(8)
        pos0 = model.position
        out = np.empty(steps, np.int64)
        _lib.check(lib.cthip_sync())
        _lib.check(lib.cthip_timer_start())
        _lib.check(lib.cthip_decoder_generate(model.handle, steps, out.ctypes.data))
        ms = C.c_float()
        _lib.check(lib.cthip_timer_stop(C.byref(ms)))
        best = min(best or 1e30, ms.value * 1e3 / steps)
    nbytes = float(np.mean([model.step_bytes(t + 1) for t in range(pos0, pos0 + steps)]))
    return best, nbytes, f"{pos0}..{pos0 + steps - 1}"


def prefill_ms(model, vocab: int, s: int):
    from caten_amd import synth
    prompt = synth.prompt(vocab, s, seed=3)
    ts = []
    for _ in range(4):
        t0 = time.perf_counter()
        model.forward(prompt, s, 0)
        ts.append(time.perf_counter() - t0)
    return min(ts) * 1e3


def measure(name: str, kind: str, prompts=(512, 2048), contexts=(16, 1900), steps: int = 64) -> dict:
    from caten_amd import _lib
    lib = _lib.init()
    max_seq = max([c + steps + 16 for c in contexts] + list(prompts) + [64])
    t0 = time.perf_counter()
    model, cfg, gflop = (llama_session if kind == "llama" else mixed_session)(name, max_seq)
    err = agree(model, cfg["vocab"])
    if not err < 2e-2:
        raise SystemExit(f"bench_mixed: {kind} {name}: prompt and decode logits differ by {err:.3g}; no figure is reported")
    print(f"# {kind} at the size of {name}: loaded and checked in {time.perf_counter() - t0:.1f} s", file=sys.stderr, flush=True)
    res = {"size": name, "model": kind, "dtype": "bf16", "data": "synthetic", "prompt_vs_decode_rel_error": err,
           "launches_per_layer": int(lib.cthip_decoder_layer_launches(model.handle)), "decode": [], "prefill": []}
    for plen in contexts:
        us, nbytes, positions = decode_us(model, lib, cfg["vocab"], plen, steps)
        gbs = nbytes / us / 1e3
        res["decode"].append({"positions": positions, "us_per_step": round(us, 1), "tokens_per_s": round(1e6 / us, 1), "bytes_per_step": int(nbytes),
                              "GBps": round(gbs, 1), "frac": round(gbs / HBM_PEAK_GBS, 4)})
    for s in prompts:
        ms = prefill_ms(model, cfg["vocab"], s)
        res["prefill"].append({"tokens": s, "ms": round(ms, 3), "tokens_per_s": round(s / ms * 1e3), "linear_TFLOPs": round(gflop * s / ms, 1)})
    model.close()
    return res


def main(names=None, kinds=("own", "llama"), **measured) -> None:
    for name in names or sizes():
        if name not in sizes():
            raise SystemExit(f"bench_mixed: unknown size {name} (known: {', '.join(sizes())})")
        for kind in kinds:
            print(json.dumps(measure(name, design_of(name) if kind == "own" else kind, **measured)), flush=True)


if __name__ == "__main__":
    ap = argparse.ArgumentParser()
    ap.add_argument("--sizes", default="")
    ap.add_argument("--kinds", default="own,llama", help="own: the size's design")
    ap.add_argument("--contexts", default="16,1900", help="prompt lengths in front of the timed decode steps")
    ap.add_argument("--prompts", default="512,2048", help="timed prompt lengths")
    ap.add_argument("--steps", type=int, default=64)
    ap.add_argument("--option", action="append", default=[], metavar="NAME=VALUE")
    a = ap.parse_args()
    from caten_amd import _lib
    for kv in a.option:
        opt, value = kv.split("=")
        _lib.check(_lib.init().cthip_set_option(opt.encode(), int(value)))
    main([n for n in a.sizes.split(",") if n], a.kinds.split(","), steps=a.steps,
         contexts=[int(c) for c in a.contexts.split(",") if c], prompts=[int(c) for c in a.prompts.split(",") if c])
