"""Mixed decoders without a GPU: model directories, configurations, the C ABI's answers before a device is there, and the
plain restatement (oracle/mixers.py) against independent formulations."""
import ctypes as C
import importlib.machinery
import importlib.util
import json
import os

import numpy as np
import pytest
import torch
import torch.nn.functional as F

from caten_amd import _lib, llm, safetensors, synth
from caten_amd.quant import from_bf16, to_bf16
from oracle import mixers
from tests import mixed_models as mm

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))


# ---- the restatement ----
def test_short_conv_is_a_causal_depthwise_convolution():
    rng = np.random.default_rng(0)
    for taps in (1, 2, 5):
        x, w = rng.standard_normal((9, 6)), rng.standard_normal((6, taps))
        want = F.silu(F.conv1d(F.pad(torch.tensor(x.T)[None], (taps - 1, 0)), torch.tensor(w)[:, None], groups=6))[0].T
        np.testing.assert_allclose(mixers.short_conv(x, w), want.numpy(), atol=1e-12)


def test_sink_is_a_key_with_a_zero_value():
    rng = np.random.default_rng(1)
    h, m = rng.standard_normal((7, 24)), dict(heads=3, dim=8, vdim=5, kv_rank=6, scale=0.4)
    cfg = mm.config([mm.latent(**m)], width=24)
    w = mm.weights(cfg, 2)
    got = mixers.latent_attention_mixer(h, m, lambda n: w["l0.mix." + n].astype(np.float64), 1e-5)
    t = {k[7:]: torch.tensor(v.astype(np.float64)) for k, v in w.items() if k.startswith("l0.mix.")}
    x = torch.tensor(h)
    c = x @ t["dkv"].T
    c = c * torch.rsqrt((c * c).mean(-1, keepdim=True) + 1e-5) * t["dkv.norm"]
    q, k, v = (x @ t["q"].T).view(7, 3, 8), (c @ t["uk"].T).view(7, 3, 8), (c @ t["uv"].T).view(7, 3, 5)
    s = torch.einsum("ihd,jhd->hij", q, k) * 0.4 + torch.full((7, 7), -torch.inf, dtype=torch.float64).triu(1)
    s = torch.cat([t["sink"][:, None, None].expand(3, 7, 1), s], -1).softmax(-1)[..., 1:]
    o = torch.einsum("hij,jhd->ihd", s, v).reshape(7, -1) * torch.sigmoid(x @ t["g"].T)
    np.testing.assert_allclose(got, (o @ t["o"].T).numpy(), atol=1e-12)


def test_delta_recurrence_against_its_chunk_form():
    """the same outputs from one triangular solve over the whole sequence"""
    rng = np.random.default_rng(3)
    T, dk, dv = 40, 6, 5
    q, k, v = mixers.unit(rng.standard_normal((T, dk))), mixers.unit(rng.standard_normal((T, dk))), rng.standard_normal((T, dv))
    g, beta = rng.uniform(0.3, 1.0, T), rng.uniform(0.0, 1.0, T)
    G = np.cumsum(np.log(g))
    D = np.exp(np.minimum(G[:, None] - G[None, :], 0.0))
    A = np.tril(beta[:, None] * D * (k @ k.T), -1)
    U = np.linalg.solve(np.eye(T) + A, beta[:, None] * v)
    want = np.tril(D * (q @ k.T)) @ U
    got, S = mixers.delta_recurrence(q, k, v, g, beta)
    np.testing.assert_allclose(got, want, atol=1e-10)
    np.testing.assert_allclose(S, (k * np.exp(G[-1] - G)[:, None]).T @ U, atol=1e-10)


def test_norms_positions_and_gates():
    rng = np.random.default_rng(4)
    x, w = rng.standard_normal((5, 12)), rng.standard_normal(12)
    tx, tw = torch.tensor(x), torch.tensor(w)
    np.testing.assert_allclose(mixers.layer_norm(x, w, 1e-3), F.layer_norm(tx, (12,), tw, None, 1e-3).numpy(), atol=1e-12)
    np.testing.assert_allclose(mixers.rms_norm(x, w, 1e-3), F.rms_norm(tx, (12,), tw, 1e-3).numpy(), atol=1e-12)
    np.testing.assert_allclose(mixers.softplus(40 * x), F.softplus(40 * tx, threshold=1e9).numpy(), atol=1e-12)
    np.testing.assert_allclose(mixers.silu(x), F.silu(tx).numpy(), atol=1e-12)
    t = mixers.sinusoid([0, 3], 6)
    assert np.array_equal(t[0], [0, 1, 0, 1, 0, 1])
    np.testing.assert_allclose(t[1], [np.sin(3), np.cos(3), np.sin(3 / 10000 ** (1 / 3)), np.cos(3 / 10000 ** (1 / 3)),
                                      np.sin(3 / 10000 ** (2 / 3)), np.cos(3 / 10000 ** (2 / 3))], atol=1e-12)


def test_rotation_is_a_complex_product():
    rng = np.random.default_rng(6)
    x, f = rng.standard_normal((5, 3, 10)), np.array([1.0, 0.3, 0.01, 2.5])
    pos = [0, 1, 7, 100, 4000]
    z = (x[..., :4] + 1j * x[..., 4:8]) * 1.2 * np.exp(1j * np.asarray(pos)[:, None, None] * f)
    got = mixers.rotate_half(x, pos, f, 1.2)
    np.testing.assert_allclose(got, np.concatenate([z.real, z.imag, x[..., 8:]], -1), atol=1e-9)


def test_yarn_frequencies():
    plain = 100.0 ** (-np.arange(0, 16, 2) / 16)
    f, m = mixers.yarn(dict(dims=16, base=100.0))
    assert m == 1.0
    np.testing.assert_allclose(f, plain, rtol=1e-14)
    f, m = mixers.yarn(dict(dims=16, base=100.0, scaling=dict(factor=1.0, original=64, fast=8.0, slow=1.0)))
    assert m == 1.0
    np.testing.assert_allclose(f, plain, rtol=1e-14)
    # pair i turns original f_i / (2 pi) times: above `fast` turns it stays, below `slow` it is divided by the factor
    f, m = mixers.yarn(dict(dims=64, base=1e4, scaling=dict(factor=4.0, original=2048, fast=32.0, slow=1.0)))
    plain = 1e4 ** (-np.arange(0, 64, 2) / 64)
    turns = 2048 * plain / (2 * np.pi)
    assert m == pytest.approx(0.1 * np.log(4.0) + 1.0)
    quotient = plain / f
    assert np.all(quotient[turns > 45] == 1.0) and np.allclose(quotient[turns < 0.7], 4.0) and np.all(np.diff(quotient) >= -1e-12)
    # the ramp is clipped at the first pair and at the last entry of the head, and may have no width
    f, _ = mixers.yarn(dict(dims=8, base=10.0, scaling=dict(factor=2.0, original=1, fast=100.0, slow=50.0)))
    np.testing.assert_allclose(f, np.r_[1.0, 10.0 ** (-np.arange(2, 8, 2) / 8) / 2], rtol=1e-14)


def test_window_attention_against_masked_softmax():
    """grouped heads, window and zero sink as one dense softmax with a column of zeros"""
    rng = np.random.default_rng(7)
    T, m = 20, mm.window(6, 2, 8, 5, 7, 0.4, 6)
    cfg = mm.matalix([mm.parallel(m, mm.lightning(1, 4, 4))], width=24)
    w = {k[12:]: v.astype(np.float64) for k, v in mm.weights(cfg, 3).items() if k.startswith("l0.mix.left.")}
    h = rng.standard_normal((T, 24))
    got = mixers.window_attention(h, m, w.__getitem__, 1e-5)
    t = {k: torch.tensor(v) for k, v in w.items()}
    x = torch.tensor(h)
    q = F.rms_norm(F.linear(x, t["q"], t["q.b"]), (48,), t["q.norm"], 1e-5).view(T, 6, 8)
    k = F.rms_norm(F.linear(x, t["k"], t["k.b"]), (16,), t["k.norm"], 1e-5).view(T, 2, 8)
    v = F.linear(x, t["v"], t["v.b"]).view(T, 2, 5)
    f, c = mixers.yarn(m["rot"])
    q, k = (torch.tensor(mixers.rotate_half(a.numpy(), range(T), f, c)) for a in (q, k))
    k, v = k.repeat_interleave(3, 1), v.repeat_interleave(3, 1)
    s = torch.einsum("ihd,jhd->hij", q, k) * 0.4
    seen = torch.ones(T, T, dtype=torch.bool).tril() & torch.ones(T, T, dtype=torch.bool).triu(-6)
    s = torch.cat([s.masked_fill(~seen, -torch.inf), torch.zeros(6, T, 1, dtype=torch.float64)], -1)
    o = torch.einsum("hij,jhd->ihd", s.softmax(-1)[..., :-1], v).reshape(T, -1) * torch.sigmoid(x @ t["g"].T)
    np.testing.assert_allclose(got, (o @ t["o"].T).numpy(), atol=1e-11)


def test_lightning_recurrence_against_its_quadratic_form():
    rng = np.random.default_rng(8)
    q, k, v = (rng.standard_normal((30, n)) for n in (6, 6, 4))
    for g in (0.0, 0.7, 1.0):
        back = np.arange(30)[:, None] - np.arange(30)[None, :]
        D = np.where(back >= 0, np.float64(g) ** np.maximum(back, 0), 0.0)
        o, S = mixers.lightning_recurrence(q, k, v, g)
        np.testing.assert_allclose(o, (D * (q @ k.T)) @ v, atol=1e-11)
        np.testing.assert_allclose(S, (k * D[-1][:, None]).T @ v, atol=1e-11)


def test_clamped_unit():
    w = {"gate": np.array([[1.0], [1.0]]), "up": np.array([[1.0], [-1.0]]), "down": np.eye(2)}
    g = np.minimum([[5.0], [-9.0]], 2.0)
    u = np.clip(np.array([[5.0, -5.0], [-9.0, 9.0]]), -2.0, 2.0)
    np.testing.assert_allclose(mixers.clamped_mlp(np.array([[5.0], [-9.0]]), 2.0, w.__getitem__), g * mixers.sigmoid(1.702 * g) * (u + 1))


# ---- model directories ----
def test_safetensors_round_trip(tmp_path):
    p = str(tmp_path / "m.safetensors")
    rng = np.random.default_rng(5)
    a = rng.standard_normal((3, 4)).astype(np.float32)
    t = {"a": ("f32", (3, 4), a), "b": ("bf16", (12,), to_bf16(a.ravel())), "c": ("i32", (2,), np.array([7, -1], np.int32)),
         "none": ("f32", (0,), np.empty(0, np.float32))}
    safetensors.write(p, t)
    got = safetensors.read(p)
    assert {k: v[:2] for k, v in got.items()} == {k: v[:2] for k, v in t.items()}
    assert np.array_equal(got["a"][2].view(np.float32).reshape(3, 4), a)
    assert np.array_equal(got["c"][2].view(np.int32), [7, -1])
    from safetensors.numpy import load_file  # the public reader takes what the writer wrote
    del t["b"]
    safetensors.write(p, t)
    assert np.array_equal(load_file(p)["a"], a)


def test_safetensors_refuses_what_does_not_fit(tmp_path):
    p = tmp_path / "m.safetensors"

    def put(header, data=b"", n=None):
        h = json.dumps(header).encode()
        p.write_bytes((len(h) if n is None else n).to_bytes(8, "little") + h + data)
    p.write_bytes(b"123")
    with pytest.raises(ValueError, match="not a safetensors"):
        safetensors.read(str(p))
    put({}, n=1000)
    with pytest.raises(ValueError, match="exceed"):
        safetensors.read(str(p))
    put({"a": {"dtype": "F32", "shape": [2], "data_offsets": [0, 8]}}, b"1234")
    with pytest.raises(ValueError, match="expected 8"):
        safetensors.read(str(p))
    put({"a": {"dtype": "F32", "shape": [1], "data_offsets": [0, 8]}}, b"12345678")
    with pytest.raises(ValueError, match="expected 4"):
        safetensors.read(str(p))
    put({"a": {"dtype": "F64", "shape": [1], "data_offsets": [0, 8]}}, b"12345678")
    with pytest.raises(ValueError, match="dtype F64"):
        safetensors.read(str(p))


def test_bf16_rounding():
    x = np.array([1.0, 1.0 + 2 ** -8, 1.0 + 3 * 2 ** -8, -1.0 - 2 ** -7, 3.4e38, 1e-40, 0.0], np.float32)
    want = torch.tensor(x).bfloat16().float().numpy()
    assert np.array_equal(from_bf16(to_bf16(x)), want)
    t = llm.Tensor.from_f32(np.arange(6, dtype=np.float32).reshape(2, 3), "bf16")
    assert (t.rows, t.cols, t.raw.size) == (2, 3, 12)


def test_configuration():
    cfg = mm.config([mm.delta(6, 3, 8, 12, 5, ff=40), mm.latent(2, 16, 24, 10, 0.5)], width=30, vocab=50, eps=1e-3, cap=7.0)
    c = llm.zuselix_config(cfg)
    assert (c["dim"], c["vocab"], c["eps"], c["logit_softcap"], c["norm"], c["position_base"]) == (30, 50, 1e-3, 7.0, "layernorm", 10000.0)
    assert c["layers"] == [dict(mixer="delta", heads=6, kv_heads=3, dim=8, vdim=12, conv=5, ffn=40),
                           dict(mixer="latent", heads=2, dim=16, vdim=24, kv_rank=10, scale=0.5, sink=True, gate=True, ffn=0)]
    bad = mm.config([mm.delta()])
    bad["layers"][0]["type"] = "window"
    with pytest.raises(ValueError, match="layer 0: mixer type 'window'"):
        llm.zuselix_config(bad)
    bad = mm.config([mm.latent(ff=8)])
    bad["layers"][0]["mlp"]["kind"] = "experts"
    with pytest.raises(ValueError, match="kind 'experts'"):
        llm.zuselix_config(bad)


def test_configuration_of_parallel_mixers():
    cfg = mm.matalix([mm.parallel(mm.window(6, 3, 10, 12, 9, 0.3, 8), mm.lightning(2, 7, 5, [0.5, 0.25]), 0.1, 0.2, ff=40, limit=1.5), mm.parallel()],
                     width=30, vocab=50, eps=1e-3, loop=dict(start=0, stop=1, times=3))
    c = llm.matalix_config(cfg)
    assert (c["dim"], c["vocab"], c["eps"], c["norm"], c["norm_plus_one"], c["tied_head"], c["loop"]) == (30, 50, 1e-3, "rmsnorm", True, True, (0, 1, 3))
    left, right = c["layers"][0]["mixers"]
    assert left == dict(mixer="window", heads=6, kv_heads=3, dim=10, vdim=12, scale=0.3, window=9, bias=True, qk_norm=True, sink="zero", gate=True,
                        out_scale=0.1, rot=dict(dims=8, base=10000.0, factor=8.0, original=64, fast=8.0, slow=1.0))
    assert right == dict(mixer="lightning", heads=2, dim=7, vdim=5, decay=[0.5, 0.25], out_scale=0.2)
    assert (c["layers"][0]["ffn"], c["layers"][0]["glu"], c["layers"][0]["layer_scale"]) == (40, (1.702, 1.5, 1.0), True)
    assert "ffn" not in c["layers"][1]
    del cfg["loop"]
    assert llm.matalix_config(cfg)["loop"] is None
    bad = mm.matalix([mm.delta()])
    with pytest.raises(ValueError, match="layer 0: mixer type 'delta'"):
        llm.matalix_config(bad)
    bad = mm.matalix([mm.parallel(ff=8)])
    bad["layers"][0]["mlp"]["kind"] = "experts"
    with pytest.raises(ValueError, match="kind 'experts'"):
        llm.matalix_config(bad)


def test_looped_layers_of_the_restatement():
    """a loop is its layers written out, with the embedding added in between"""
    layers = [mm.parallel(ff=8), mm.parallel(mm.window(2, 1, 8, 8, 5)), mm.parallel()]
    cfg = mm.matalix(layers, width=16, vocab=20, loop=dict(start=1, stop=3, times=2))
    w, toks = mm.weights(cfg, 4), mm.tokens(cfg, 12)
    logits, stream = mixers.matalix(cfg, w, toks)
    assert stream.shape == (5, 12, 16)
    t = {k: v.astype(np.float64) for k, v in w.items()}
    x0 = x = t["embed"][toks]
    for step in (0, 1, 2, None, 1, 2):
        if step is None:
            x = x + x0
            continue
        one = dict(cfg, layers=[layers[step]], loop=None)
        rest = {k.replace(f"l{step}.", "l0.", 1): v for k, v in t.items() if k.startswith(f"l{step}.")}
        # the layer as a model of its own whose embedding table holds the stream
        x = mixers.matalix(one, dict(rest, embed=x, **{"final.norm": t["final.norm"]}), range(12))[1][0]
    np.testing.assert_allclose(stream[-1], x, atol=1e-10)
    np.testing.assert_allclose(logits, mixers.rms_norm(x, 1 + t["final.norm"], 1e-5) @ t["embed"].T, atol=1e-9)


def test_registry(tmp_path):
    (tmp_path / "config.json").write_text(json.dumps({"architecture": "Other"}))
    with pytest.raises(ValueError, match="'Other' is not registered .known: Matalix, Zuselix"):
        llm.load_model(str(tmp_path))
    (tmp_path / "config.json").write_text(json.dumps(mm.config([mm.delta()])))
    with pytest.raises(ValueError, match="dtype 'int8'"):
        llm.load_model(str(tmp_path), "int8")


def test_shapes_of_the_measured_sizes():
    for name, cfg in synth.ZUSELIX_CONFIGS.items():
        shapes = synth.zuselix_shapes(cfg)
        assert shapes["l2.mix.uk"] == (cfg["layers"][2]["mixer"]["heads"] * 128, 512) and "l0.mix.A_log" in shapes, name
    for name, cfg in synth.MATALIX_CONFIGS.items():
        shapes, left = synth.matalix_shapes(cfg), cfg["layers"][0]["mixer"]["left"]
        assert shapes["l3.mix.left.q"] == shapes["l3.mix.left.o"][::-1] == (left["heads"] * 128, cfg["width"]) and "head" not in shapes, name
    import bench_mixed
    assert sum(bench_mixed.layer_runs(synth.MATALIX_CONFIGS["matalix-1b"])) == 22
    assert sum(bench_mixed.layer_runs(synth.ZUSELIX_CONFIGS["zuselix-1b"])) == 21


def test_c_abi_before_a_device_is_there():
    lib = _lib.load()
    if _lib.is_initialised():
        pytest.skip("the library is initialised in this process")
    h, cfg, layers = C.c_void_p(), _lib.MixedConfig(), (_lib.LayerSpec * 1)()
    assert lib.cthip_decoder_create_mixed(C.byref(h), C.byref(cfg), layers) == _lib.E_NOT_INIT
    tok = C.c_int64()
    assert lib.cthip_decoder_forward_rows(None, None, 1, 0, None, 0, C.byref(tok), None) == _lib.E_NOT_INIT


# ---- the replay program's bookkeeping, over a stand-in session ----
class Recorder:
    def __init__(self):
        self.calls = []

    def forward_rows(self, tokens, rows, n):
        self.calls.append((list(tokens), list(rows), n))
        return 0, np.full((len(rows), 3), float(len(self.calls)), np.float32)


def trace_run():
    loader = importlib.machinery.SourceFileLoader("trace_run", os.path.join(ROOT, "bin", "trace_run"))
    mod = importlib.util.module_from_spec(importlib.util.spec_from_loader("trace_run", loader))
    loader.exec_module(mod)
    return mod


def test_replay_follows_requests(tmp_path):
    m = Recorder()
    r = trace_run().Replay(m, str(tmp_path))

    def step(i, rid, toks, want, end=()):
        r.step({"step": i, "entries": [{"id": rid, "tokens": toks, "want": want}], "end": list(end)})
    step(0, "a", [1, 2, 3], [2])
    step(1, "a", [4], [], ["a"])
    step(2, "b", [5, 6], [0, 1], ["b"])
    step(3, "a", [7], [0])  # a name used again is a new request
    assert m.calls == [([1, 2, 3], [2], 0), ([4], [], 3), ([5, 6], [0, 1], 0), ([7], [0], 0)]
    assert sorted(p.name for p in tmp_path.iterdir()) == ["0.f32", "2.f32", "3.f32"]
    assert np.array_equal(np.fromfile(tmp_path / "2.f32", "<f4"), [3.0] * 6)
    with pytest.raises(ValueError, match="before a has ended"):
        step(4, "c", [1], [])
    with pytest.raises(ValueError, match="no tokens"):
        step(5, "a", [], [])
