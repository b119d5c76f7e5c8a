"""Decoder front-end: mirrors `make-gpt2` / `gpt2-generate` (apps/gpt2/gpt2.lisp:82-113)
and the Transformer it compiles (external/llm/layers.lisp:73-90) on top of the
device-resident decoder session of libcaten_hip.so.

    model = make_gpt2(cfg, state_dict)           # state dict: reference keys -> (kind, raw GGUF bytes, shape)
    tok = model.forward(x=[...], s=len, n=start) # one compiled-graph `forward`
    toks = gpt2_generate(model, prompt_ids, max_length=100)
"""
from __future__ import annotations

import ctypes as C
import json
import os
from typing import Dict, List, Optional, Sequence, Tuple

import numpy as np

from . import _lib, safetensors
from .quant import from_bf16, packed_nbytes, quantize, to_bf16

# *remap-key* (apps/gpt2/gpt2.lisp:52-70): GGUF tensor names -> Caten state-dict keys
GPT2_REMAP = [
    ("blk.", "h."), ("token_embd.weight", "wte.weight"), ("position_embd.weight", "wpe.weight"),
    (".attn_norm.weight", ".ln_1.affine"), (".attn_norm.bias", ".ln_1.bias"),
    (".attn_qkv.weight", ".attn.c_attn.weight"), (".attn_qkv.bias", ".attn.c_attn.bias"),
    (".ffn_down.weight", ".mlp.c_proj.weight"), (".ffn_down.bias", ".mlp.c_proj.bias"),
    (".ffn_norm.weight", ".ln_2.affine"), (".ffn_norm.bias", ".ln_2.bias"),
    (".ffn_up.weight", ".mlp.c_fc.weight"), (".ffn_up.bias", ".mlp.c_fc.bias"),
    (".attn_output.weight", ".attn.c_proj.weight"), (".attn_output.bias", ".attn.c_proj.bias"),
    ("output.weight", "lm_head.weight"), ("output_norm.bias", "ln_f.bias"), ("output_norm.weight", "ln_f.affine"),
]


def remap_key(key: str) -> str:
    for before, after in GPT2_REMAP:
        key = key.replace(before, after)
    return key


class Tensor:
    """One state-dict entry as it sits in a GGUF file: type, raw bytes, (rows, cols)."""

    def __init__(self, kind: str, raw: np.ndarray, rows: int, cols: int):
        self.kind, self.rows, self.cols = kind, int(rows), int(cols)
        self.raw = np.ascontiguousarray(np.asarray(raw).view(np.uint8).ravel())
        want = packed_nbytes(kind, self.rows * self.cols)
        if self.raw.size != want:
            raise ValueError(f"Tensor: {self.raw.size} bytes for a {kind} ({rows},{cols}) tensor, expected {want}")

    @classmethod
    def from_f32(cls, a: np.ndarray, kind: str = "f32") -> "Tensor":
        a = np.ascontiguousarray(a, np.float32)
        rows, cols = (a.shape if a.ndim == 2 else (1, a.size))
        if kind == "f32":
            return cls(kind, a.view(np.uint8), rows, cols)
        if kind == "f16":
            return cls(kind, a.astype(np.float16).view(np.uint8), rows, cols)
        if kind == "bf16":
            return cls(kind, to_bf16(a).view(np.uint8), rows, cols)
        return cls(kind, quantize(kind, a), rows, cols)


def gpt2_state_dict(weights: dict, linear_kind: str = "f32") -> Dict[str, Tensor]:
    """Synthetic weights (caten_amd.synth.gpt2_weights) -> state dict under the reference's keys.
    Linear weights are stored as `linear_kind`; embeddings, LayerNorm and biases stay fp32."""
    sd = {"wte.weight": Tensor.from_f32(weights["wte"]), "wpe.weight": Tensor.from_f32(weights["wpe"]),
          "ln_f.affine": Tensor.from_f32(weights["lnf_g"]), "ln_f.bias": Tensor.from_f32(weights["lnf_b"]),
          "lm_head.weight": Tensor.from_f32(weights["lm_head"], linear_kind)}
    names = {"ln1_g": "ln_1.affine", "ln1_b": "ln_1.bias", "attn_w": "attn.c_attn.weight", "attn_b": "attn.c_attn.bias",
             "proj_w": "attn.c_proj.weight", "proj_b": "attn.c_proj.bias", "ln2_g": "ln_2.affine", "ln2_b": "ln_2.bias",
             "fc_w": "mlp.c_fc.weight", "fc_b": "mlp.c_fc.bias", "fc2_w": "mlp.c_proj.weight", "fc2_b": "mlp.c_proj.bias"}
    for src, dst in names.items():
        for l, a in enumerate(weights[src]):
            sd[f"h.{l}.{dst}"] = Tensor.from_f32(a, linear_kind if src.endswith("_w") else "f32")
    return sd


def llama_state_dict(weights: dict, linear_kind: str = "f32", threads: int = 1) -> Dict[str, Tensor]:
    """`threads` > 1 quantises the tensors on a thread pool (NumPy releases the interpreter lock inside its loops)."""
    names = {"attn_norm": "attention_norm.weight", "ffn_norm": "ffn_norm.weight", "wq": "attention.wq.weight",
             "wk": "attention.wk.weight", "wv": "attention.wv.weight", "wo": "attention.wo.weight",
             "w_gate": "feed_forward.w1.weight", "w_down": "feed_forward.w2.weight", "w_up": "feed_forward.w3.weight"}
    jobs = [("tok_embeddings.weight", weights["tok_emb"], "f32"), ("norm.weight", weights["norm_w"], "f32"),
            ("output.weight", weights["lm_head"], linear_kind)]
    for src, dst in names.items():
        for l, a in enumerate(weights[src]):
            jobs.append((f"layers.{l}.{dst}", a, linear_kind if src.startswith("w") else "f32"))
    if threads > 1:
        from concurrent.futures import ThreadPoolExecutor
        with ThreadPoolExecutor(threads) as pool:
            tensors = list(pool.map(lambda j: Tensor.from_f32(j[1], j[2]), jobs))
    else:
        tensors = [Tensor.from_f32(a, kind) for _, a, kind in jobs]
    return {key: t for (key, _, _), t in zip(jobs, tensors)}


class Transformer:
    """The compiled Transformer graph: `forward(x, s, n)` as apps/gpt2/gpt2.lisp:104 calls it."""

    def __init__(self, cfg: dict, arch: str = "gpt2", device: int = 0):
        self.cfg = dict(cfg)
        self.arch = arch
        self.lib = _lib.init(device)
        self.handle = C.c_void_p()
        self._create(cfg)

    def _create(self, cfg: dict) -> None:
        arch = self.arch
        c = _lib.DecoderConfig()
        c.arch = _lib.ARCH_GPT2 if arch == "gpt2" else _lib.ARCH_LLAMA
        c.n_layers, c.dim, c.n_heads = cfg["n_layers"], cfg["dim"], cfg["n_heads"]
        c.n_kv_heads = cfg.get("n_kv_heads", cfg["n_heads"])
        c.ffn, c.vocab, c.max_seq = cfg["ffn"], cfg["vocab"], cfg["max_seq"]
        c.eps = cfg.get("eps", 1e-5)
        c.rope_base = cfg.get("rope_base", 10000.0)
        _lib.check(self.lib.cthip_decoder_create(C.byref(self.handle), C.byref(c)))

    def load_state_dict(self, sd: Dict[str, Tensor]) -> "Transformer":
        """load-state-dict (source/api/module.lisp:290-320)"""
        for key, t in sd.items():
            _lib.check(self.lib.cthip_decoder_load(self.handle, key.encode(), _lib.GGML_TYPE[t.kind], t.raw.ctypes.data,
                                                   t.rows, t.cols))
        missing = self.lib.cthip_decoder_missing(self.handle)
        if missing:
            raise _lib.HipError(-5, f"load-state-dict: {missing} tensors of the model are missing from the state dict")
        return self

    def forward(self, x: Sequence[float], s: Optional[int] = None, n: int = 0, return_logits: bool = False):
        """(forward model `(x . tokens) `(s . len) `(n . start-pos)) -> greedy token of the last position."""
        toks = np.ascontiguousarray(x, np.float32).ravel()
        s = toks.size if s is None else s
        if s != toks.size:
            raise ValueError(f"forward: s = {s} but x holds {toks.size} tokens")
        tok = C.c_int64()
        logits = np.empty(self.cfg["vocab"], np.float32) if return_logits else None
        _lib.check(self.lib.cthip_decoder_forward(self.handle, toks.ctypes.data, s, n, C.byref(tok),
                                                  logits.ctypes.data if return_logits else None))
        return (int(tok.value), logits) if return_logits else int(tok.value)

    def forward_rows(self, x: Sequence[float], rows: Sequence[int], n: int = 0) -> Tuple[int, np.ndarray]:
        """forward, with the logits of the listed positions of x: (greedy token of the last one, (len(rows), vocab))"""
        toks = np.ascontiguousarray(x, np.float32).ravel()
        idx = np.ascontiguousarray(rows, np.int32).ravel()
        out = np.empty((idx.size, self.cfg["vocab"]), np.float32)
        tok = C.c_int64()
        _lib.check(self.lib.cthip_decoder_forward_rows(self.handle, toks.ctypes.data, toks.size, n,
                                                       idx.ctypes.data_as(C.POINTER(C.c_int)), idx.size, C.byref(tok),
                                                       out.ctypes.data))
        return int(tok.value), out

    def generate_until(self, max_steps: int, eos_token: int) -> List[int]:
        """Greedy tokens from the device-resident loop until `eos_token` has been produced (it is the last element)
        or `max_steps` tokens exist; the stop condition is evaluated on the device."""
        out = np.empty(max(max_steps, 1), np.int64)
        n = C.c_int()
        _lib.check(self.lib.cthip_decoder_generate_until(self.handle, max_steps, int(eos_token), out.ctypes.data, C.byref(n)))
        return [int(t) for t in out[:n.value]]

    def generate_on_device(self, steps: int) -> List[int]:
        """Continues greedily for `steps` tokens without returning to the host in between."""
        out = np.empty(max(steps, 1), np.int64)
        _lib.check(self.lib.cthip_decoder_generate(self.handle, steps, out.ctypes.data))
        return [int(t) for t in out[:steps]]

    @property
    def position(self) -> int:
        return int(self.lib.cthip_decoder_position(self.handle))

    def step_bytes(self, t: int) -> int:
        return int(self.lib.cthip_decoder_step_bytes(self.handle, t))

    def peek(self, what: str) -> np.ndarray:
        p, n = C.c_void_p(), C.c_int64()
        _lib.check(self.lib.cthip_decoder_peek(self.handle, what.encode(), C.byref(p), C.byref(n)))
        out = np.empty(n.value, np.float32)
        _lib.check(self.lib.cthip_d2h(out.ctypes.data, p.value, out.nbytes))
        return out

    def close(self):
        if self.handle:
            self.lib.cthip_decoder_destroy(self.handle)
            self.handle = None

    def __del__(self):
        try:
            self.close()
        except Exception:
            pass


def make_gpt2(cfg: dict, state_dict: Dict[str, Tensor], device: int = 0) -> Transformer:
    """make-gpt2 (apps/gpt2/gpt2.lisp:82-93) minus the download: build the Transformer, load the state dict."""
    return Transformer(cfg, "gpt2", device).load_state_dict(state_dict)


def make_llama(cfg: dict, state_dict: Dict[str, Tensor], device: int = 0) -> Transformer:
    return Transformer(cfg, "llama", device).load_state_dict(state_dict)


class MixedTransformer(Transformer):
    """A decoder whose layers are listed one by one (cthip_decoder_create_mixed).  cfg: `vocab`, `dim`, `max_seq`, `eps`,
    `norm` ("layernorm" or "rmsnorm"), `norm_plus_one` (norm weights stored around zero), `position_base`, `logit_softcap`
    (0 = none), `tied_head`, `loop` ((start, stop, times) of the layers that run several times, None = none), `precision`
    (operand format of the products over several rows, None = the library's option) and `layers`, each a dict of `mixer`
    ("delta", "latent", "window" or "lightning") and that mixer's sizes, or `mixers`, a list of two such dicts side by
    side, and of `ffn` (0 = none), `glu` ((alpha, limit, shift) of the gated unit, None = SwiGLU) and `layer_scale`.
    A window mixer's `rot`: None or a dict of `dims`, `base` and, for YaRN, `factor`, `original`, `fast`, `slow`; its
    `sink`: None, "tensor" or "zero".  A lightning mixer's `decay`: one factor per head."""

    MIXERS = {"delta": _lib.MIXER_DELTA, "latent": _lib.MIXER_LATENT, "window": _lib.MIXER_WINDOW, "lightning": _lib.MIXER_LIGHTNING}
    SINKS = {None: _lib.SINK_NONE, False: _lib.SINK_NONE, True: _lib.SINK_TENSOR, "tensor": _lib.SINK_TENSOR, "zero": _lib.SINK_ZERO}
    NORMS = {"layernorm": _lib.PRO_LAYERNORM, "rmsnorm": _lib.PRO_RMSNORM}

    def __init__(self, cfg: dict, device: int = 0):
        super().__init__(cfg, "mixed", device)

    def _create(self, cfg: dict) -> None:
        c = _lib.MixedConfig()
        c.n_layers, c.dim, c.vocab, c.max_seq = len(cfg["layers"]), cfg["dim"], cfg["vocab"], cfg["max_seq"]
        c.norm, c.eps = self.NORMS[cfg.get("norm", "layernorm")], cfg["eps"]
        c.position_base, c.logit_softcap = cfg.get("position_base") or 0.0, cfg.get("logit_softcap") or 0.0
        c.precision = -1 if cfg.get("precision") is None else cfg["precision"]
        c.norm_plus_one, c.tied_head = int(cfg.get("norm_plus_one", False)), int(cfg.get("tied_head", False))
        c.loop_start, c.loop_stop, c.loop_times = cfg.get("loop") or (0, 0, 1)
        layers = (_lib.LayerSpec * len(cfg["layers"]))()
        for y, l in zip(layers, cfg["layers"]):
            mixers = l.get("mixers") or [l]
            if len(mixers) > 2:
                raise ValueError(f"a layer has one mixer or two side by side, not {len(mixers)}")
            y.n_mixers, y.ffn = len(mixers), l.get("ffn") or 0
            y.glu_alpha, y.glu_limit, y.glu_shift = l.get("glu") or (1.0, float("inf"), 0.0)
            y.layer_scale = int(l.get("layer_scale", False))
            for s, m in zip(y.mixers, mixers):
                self._mixer(s, m)
        _lib.check(self.lib.cthip_decoder_create_mixed(C.byref(self.handle), C.byref(c), layers))

    def _mixer(self, s, m: dict) -> None:
        s.mixer, s.heads, s.dim, s.vdim = self.MIXERS[m["mixer"]], m["heads"], m["dim"], m["vdim"]
        s.kv_heads, s.conv = m.get("kv_heads", m["heads"]), m.get("conv", 0)
        s.kv_rank, s.scale = m.get("kv_rank", 0), m.get("scale", 0.0)
        s.sink, s.gate = self.SINKS[m.get("sink")], int(m.get("gate", False))
        s.window, s.bias, s.qk_norm = m.get("window", 0), int(m.get("bias", False)), int(m.get("qk_norm", False))
        s.out_scale = m.get("out_scale", 1.0)
        rot = m.get("rot")
        if rot:
            s.rot_dims, s.rot_base = rot["dims"], rot["base"]
            s.rot_factor, s.rot_original = rot.get("factor", 0.0), rot.get("original", 0.0)
            s.rot_fast, s.rot_slow = rot.get("fast", 0.0), rot.get("slow", 0.0)
        if m["mixer"] == "lightning":
            if len(m["decay"]) != m["heads"]:
                raise ValueError(f"{len(m['decay'])} decays for {m['heads']} heads")
            s.decay = (C.c_double * m["heads"])(*m["decay"])  # (the structure keeps it alive)


def zuselix_config(config: dict) -> dict:
    """config.json of a Zuselix model -> MixedTransformer's cfg (without max_seq)"""
    layers = []
    for i, l in enumerate(config["layers"]):
        m = dict(l["mixer"])
        mlp = l.get("mlp")
        if mlp is not None and mlp.get("kind", "dense") != "dense":
            raise ValueError(f"layer {i}: a feed-forward of kind {mlp['kind']!r} is not part of this design")
        m["ffn"] = int(mlp["ff"]) if mlp is not None else 0
        if l["type"] == "delta":
            m["mixer"] = "delta"
        elif l["type"] == "latent_attention":
            m.update(mixer="latent", sink=True, gate=True)
        else:
            raise ValueError(f"layer {i}: mixer type {l['type']!r} is not part of this design")
        layers.append(m)
    return dict(vocab=config["vocab"], dim=config["width"], eps=config["norm"]["eps"], norm="layernorm", position_base=10000.0,
                logit_softcap=config.get("logit_softcap") or 0.0, layers=layers)


def matalix_config(config: dict) -> dict:
    """config.json of a Matalix model -> MixedTransformer's cfg (without max_seq)"""
    layers = []
    for i, l in enumerate(config["layers"]):
        if l["type"] != "parallel":
            raise ValueError(f"layer {i}: mixer type {l['type']!r} is not part of this design")
        m, mlp = l["mixer"], l.get("mlp")
        left = {k: m["left"][k] for k in ("heads", "kv_heads", "dim", "vdim", "scale")}
        rot = m["left"]["rot"]
        left.update(mixer="window", window=m["left"]["mask"]["size"], rot=dict(dims=rot["dims"], base=rot["base"], **(rot.get("scaling") or {})),
                    bias=True, qk_norm=True, sink="zero", gate=True, out_scale=m["left_scale"])
        right = {k: m["right"][k] for k in ("heads", "dim", "vdim", "decay")}
        right.update(mixer="lightning", out_scale=m["right_scale"])
        layer = dict(mixers=[left, right], layer_scale=True)
        if mlp is not None:
            if mlp.get("kind", "dense") != "dense":
                raise ValueError(f"layer {i}: a feed-forward of kind {mlp['kind']!r} is not part of this design")
            layer.update(ffn=int(mlp["ff"]), glu=(1.702, mlp["limit"], 1.0))
        layers.append(layer)
    loop = config.get("loop")
    return dict(vocab=config["vocab"], dim=config["width"], eps=config["norm"]["eps"], norm="rmsnorm", norm_plus_one=True, tied_head=True,
                loop=(loop["start"], loop["stop"], loop["times"]) if loop else None, layers=layers)


# architecture name of a model directory's config.json -> (its configuration, the session's class)
ARCHITECTURES = {"Matalix": (matalix_config, MixedTransformer), "Zuselix": (zuselix_config, MixedTransformer)}


def load_model(path: str, dtype: str = "bfloat16", max_seq: int = 2048, device: int = 0) -> Transformer:
    """A model directory (config.json, model.safetensors) -> a session with its weights loaded.  dtype "bfloat16" keeps the
    Linear weights in 16 bits as they are; "float32" widens them and multiplies fp32 operands everywhere."""
    with open(os.path.join(path, "config.json")) as f:
        config = json.load(f)
    name = config.get("architecture")
    if name not in ARCHITECTURES:
        raise ValueError(f"{path}: architecture {name!r} is not registered (known: {', '.join(sorted(ARCHITECTURES))})")
    if dtype not in ("bfloat16", "float32"):
        raise ValueError(f"load_model: dtype {dtype!r} (bfloat16 or float32)")
    to_cfg, cls = ARCHITECTURES[name]
    cfg = dict(to_cfg(config), max_seq=max_seq)
    if dtype == "float32":
        cfg["precision"] = 0
    tensors = safetensors.read(os.path.join(path, "model.safetensors"))
    return cls(cfg, device).load_state_dict(safetensors_state_dict(tensors, widen=dtype == "float32"))


def safetensors_state_dict(tensors: dict, widen: bool = False) -> Dict[str, Tensor]:
    """tensors as safetensors.read gives them -> state dict; `widen`: bf16 values as fp32"""
    sd = {}
    for key, (kind, shape, raw) in tensors.items():
        rows, cols = shape if len(shape) == 2 else (1, int(np.prod(shape)))
        if widen and kind == "bf16":
            kind, raw = "f32", from_bf16(np.ascontiguousarray(raw))
        sd[key] = Tensor(kind, raw, rows, cols)
    return sd


def gpt2_generate(model: Transformer, prompt: Sequence[int], max_length: int = 100, on_device: bool = True,
                  keep_logits: bool = False):
    """gpt2-generate (apps/gpt2/gpt2.lisp:97-113): `max_length` forwards, the first over the whole
    prompt (prefill), each of the rest over the one new token.  With on_device the single-token
    forwards run back to back on the GPU and their tokens are read once at the end; otherwise every
    step returns its token to the host, as the reference's loop does."""
    tokens = [int(t) for t in prompt]
    out: List[int] = []
    logs = []
    if max_length <= 0:
        return (out, logs) if keep_logits else out
    if on_device and not keep_logits:
        tok = model.forward([float(t) for t in tokens], len(tokens), 0)
        out.append(tok)
        out.extend(model.generate_on_device(max_length - 1))
        return out
    start = 0
    for _ in range(max_length):
        chunk = tokens[start:]
        r = model.forward([float(t) for t in chunk], len(chunk), start, return_logits=keep_logits)
        tok = r[0] if keep_logits else r
        if keep_logits:
            logs.append(r[1])
        start = len(tokens)
        tokens.append(tok)
        out.append(tok)
    return (out, logs) if keep_logits else out


def gpt2_generate_text(model: Transformer, tokenizer, text: str, max_length: int = 100, on_device: bool = True,
                       expected: Optional[str] = None) -> str:
    """gpt2-generate with its string interface (apps/gpt2/gpt2.lisp:97-113): encode the input, run `max_length`
    greedy forwards, decode prompt + generated tokens; `expected` asserts the decoded text as the reference's
    keyword does."""
    if not isinstance(text, str):
        raise TypeError("gpt2_generate_text: input must be a string")
    prompt = tokenizer.encode(text)
    if not prompt:
        raise ValueError("gpt2_generate_text: the input encodes to no tokens")
    decoded = tokenizer.decode(prompt + gpt2_generate(model, prompt, max_length, on_device=on_device))
    if expected is not None and decoded != expected:
        raise AssertionError(f"Expected output: {expected}, but got: {decoded}")
    return decoded
