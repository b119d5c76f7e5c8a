"""Mixed decoders (gated delta rule, latent attention) against the plain float64 restatement in oracle/mixers.py."""
import numpy as np
import pytest

from oracle import mixers
from tests import mixed_models as mm

pytestmark = pytest.mark.gpu

# fp32 sessions: summation order and a few ulp of the elementary functions.  bf16 sessions: the weights are the oracle's
# exactly, products over several rows drop 2^-16 of a product
TOL = {"float32": 2e-5, "bfloat16": 4e-4}


def all_rows(model, toks, cuts):
    out, n = [], 0
    for c in cuts:
        out.append(model.forward_rows(toks[n:n + c], range(c), n)[1])
        n += c
    assert n == len(toks)
    return np.concatenate(out)


def error(got, want):
    return np.abs(got - want).max() / np.sqrt((want ** 2).mean())


def check(cfg, w, toks, cuts, dtype="float32", max_seq=256, tol=None):
    want, _ = mixers.zuselix(cfg, w, toks)
    m = mm.session(cfg, w, dtype, max_seq)
    got = all_rows(m, toks, cuts)
    m.close()
    e = error(got, want)
    assert e < (tol or TOL[dtype]), (e, np.abs(got - want).max(1) / np.sqrt((want ** 2).mean()))


MODELS = {
    "delta": mm.config([mm.delta()]),
    "delta_mlp": mm.config([mm.delta(ff=192)]),
    "latent": mm.config([mm.latent()]),
    "latent_mlp": mm.config([mm.latent(ff=160)]),
    "stack": mm.config([mm.latent(ff=96), mm.delta(), mm.delta(ff=224), mm.latent()]),
}


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", list(MODELS))
def test_prompt_in_one_forward(name, dtype):
    cfg = MODELS[name]
    check(cfg, mm.weights(cfg, 1), mm.tokens(cfg, 75), [75], dtype)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", list(MODELS))
def test_token_by_token(name, dtype):
    cfg = MODELS[name]
    check(cfg, mm.weights(cfg, 2), mm.tokens(cfg, 40), [1] * 40, dtype)


# sizes that are multiples of nothing, single heads, shared and unshared key heads, one to many taps, wide latents
ODD = {
    "taps1_heads_unshared": mm.config([mm.delta(3, 3, 24, 40, 1), mm.latent(3, 24, 40, 20, 0.31, 88)], width=96, vocab=301),
    "one_head_each": mm.config([mm.delta(1, 1, 8, 5, 2, 50), mm.latent(1, 12, 7, 9, 1.0)], width=64, vocab=33),
    "key_head_of_six": mm.config([mm.delta(6, 1, 48, 80, 7), mm.latent(5, 80, 24, 96, 0.07, 130)], width=176),
    "wide_heads": mm.config([mm.delta(2, 1, 256, 256, 3), mm.latent(2, 256, 256, 272, 0.06)], width=256),
    "narrow_values": mm.config([mm.delta(4, 2, 200, 16, 4), mm.latent(4, 192, 16, 64, 0.07)], width=128),
    "wide_values": mm.config([mm.delta(4, 4, 16, 200, 4), mm.latent(4, 20, 160, 64, 0.2)], width=128),
    "many_heads": mm.config([mm.delta(20, 5, 16, 16, 4), mm.latent(35, 16, 16, 32, 0.3, 64)], width=160),
    "big_latent": mm.config([mm.latent(3, 32, 32, 520, 0.2), mm.latent(2, 16, 16, 1000, 0.2)], width=128),
    "width_not_16": mm.config([mm.delta(2, 1, 16, 16, 4, 72), mm.latent(2, 16, 16, 24, 0.2, 36)], width=104),
    "width_not_8": mm.config([mm.delta(2, 1, 16, 16, 4, 30), mm.latent(2, 16, 16, 24, 0.2, 27)], width=90),
    "width_odd": mm.config([mm.delta(2, 1, 16, 16, 4, 31), mm.latent(2, 16, 16, 24, 0.2)], width=77, vocab=65),
    "large_eps_and_no_cap": mm.config([mm.delta(), mm.latent()], eps=0.05, cap=None),
    "small_cap": mm.config([mm.delta(), mm.latent()], cap=1.5),
}


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", list(ODD))
def test_sizes(name, dtype):
    """a prompt, portions and single tokens, on sizes that exercise padding and every fallback"""
    cfg = ODD[name]
    check(cfg, mm.weights(cfg, 3), mm.tokens(cfg, 60), [33, 2, 9, 1, 1, 14], dtype)


@pytest.mark.parametrize("cuts", [[100], [2] * 50, [3] * 33 + [1], [7] * 14 + [2], [8] * 12 + [4], [31, 32, 33, 4], [1, 64, 35], [65, 35],
                                  [15, 16, 17, 52]])
def test_portions(cuts):
    """however the tokens are cut, the logits are those of the whole sequence"""
    cfg = MODELS["stack"]
    check(cfg, mm.weights(cfg, 4), mm.tokens(cfg, 100), cuts)


@pytest.mark.parametrize("taps", [1, 2, 5, 9])
def test_history_of_the_convolutions(taps):
    """portions shorter than the taps: the history is read and rewritten across several of them"""
    cfg = mm.config([mm.delta(conv=taps)])
    check(cfg, mm.weights(cfg, 5, conv=2.0), mm.tokens(cfg, 40), [1, 2, 1, 3, 8, 1, 2, 9, 1, 4, 8])


def test_sequences_one_after_another():
    """a sequence that starts at position 0 sees nothing of the ones before it, whatever their length"""
    cfg = MODELS["stack"]
    w = mm.weights(cfg, 6)
    m = mm.session(cfg, w)
    for seed, cuts in enumerate([[90], [1, 1, 1], [20, 1, 1], [2], [50, 2, 9], [1] * 12, [8]]):
        toks = mm.tokens(cfg, sum(cuts), seed)
        assert error(all_rows(m, toks, cuts), mixers.zuselix(cfg, w, toks)[0]) < TOL["float32"], seed
    m.close()


def test_state_does_not_go_back():
    cfg = MODELS["delta"]
    m = mm.session(cfg, mm.weights(cfg, 6))
    from caten_amd._lib import HipError
    with pytest.raises(HipError, match="starts there or at 0"):
        m.forward_rows([1, 2], [0], 3)
    m.forward_rows(list(range(12)), [], 0)
    for n in (11, 13):
        with pytest.raises(HipError, match="starts there or at 0"):
            m.forward_rows([1], [0], n)
    with pytest.raises(HipError, match="row 2"):
        m.forward_rows([1, 2], [2], 12)
    m.forward_rows([1], [0], 12)
    m.close()


def far_key_model(sink):
    """one latent layer in which token 1 asks for token 2: its query and that token's key stand out of the rest"""
    cfg = mm.config([mm.latent(heads=2, dim=16, vdim=16, kv_rank=32, scale=0.25)], width=64, vocab=200)
    w = mm.weights(cfg, 8)
    rng = np.random.default_rng(9)
    dq, dk = rng.standard_normal((2, 64)).astype(np.float32)
    w["embed"][1] = np.round(6 * dq * 8) / 8
    w["embed"][2] = np.round(6 * dk * 8) / 8

    def normed(e):
        return (e - e.mean()) / e.std()
    # q reads the direction of token 1, the latent that of token 2
    a, b = normed(w["embed"][1]), normed(w["embed"][2])
    latent_dir = rng.standard_normal(32).astype(np.float32)
    w["l0.mix.dkv"] = w["l0.mix.dkv"] * 2 + np.outer(latent_dir, b) / 16
    head = rng.standard_normal(32).astype(np.float32)
    w["l0.mix.q"] = w["l0.mix.q"] * 0.3 + np.outer(head, a) / 40
    w["l0.mix.o"] *= 8
    w["l0.mix.uk"] = w["l0.mix.uk"] * 0.3 + np.outer(head, latent_dir) / 16
    w["l0.mix.sink"][:] = sink
    from caten_amd.quant import from_bf16, to_bf16
    return cfg, {k: from_bf16(to_bf16(v.astype(np.float32).ravel())).reshape(v.shape) for k, v in w.items()}


@pytest.mark.parametrize("sink", [-4.0, 12.0, 30.0])
@pytest.mark.parametrize("at", [0, 15, 16, 31, 32, 300, 511, 512])
def test_far_key(at, sink):
    """one key among hundreds carries the softmax: at tile borders, at the first position, far behind; asked for by a
    prompt's row and by a decoded token; with a sink that is nothing, one among them, and nearly everything"""
    cfg, w = far_key_model(sink)
    toks = [3 + t % 190 for t in mm.tokens(cfg, 560)]
    toks[at] = 2
    toks[530] = toks[540] = toks[559] = 1
    want, _ = mixers.zuselix(cfg, w, toks)
    without = list(toks)
    without[at] = 7
    blind, _ = mixers.zuselix(cfg, w, without)
    seen = np.abs(want[559] - blind[559]).max() / np.sqrt((want ** 2).mean())
    assert seen > 0.5 or sink == 30.0, seen  # (the key shows in the logits)
    for dtype in ("float32", "bfloat16"):
        m = mm.session(cfg, w, dtype, 576)
        got = all_rows(m, toks, [535, 20] + [1] * 5)
        m.close()
        assert error(got, want) < TOL[dtype], dtype


@pytest.mark.parametrize("n", [1, 2, 15, 16, 17, 63, 64, 65, 255, 256, 257, 1023, 1024, 1025])
def test_decode_at_tile_and_range_borders(n):
    """the first decoded tokens behind prompts that end around the borders of key tiles and key ranges"""
    cfg = mm.config([mm.latent(heads=3, dim=16, vdim=16, kv_rank=40, scale=0.3), mm.delta(2, 1, 16, 16)], width=64, vocab=100)
    w = mm.weights(cfg, 10, q=2.0)
    toks = mm.tokens(cfg, n + 3)
    check(cfg, w, toks, [n, 1, 1, 1], max_seq=1100)


def test_first_tokens_and_the_sink():
    """with one visible key the sink decides how much of its value passes"""
    cfg = mm.config([mm.latent()])
    for sink in (-30.0, 0.0, 6.0):
        w = mm.weights(cfg, 11)
        w["l0.mix.sink"][:] = sink
        check(cfg, w, mm.tokens(cfg, 9), [1] * 9)
        check(cfg, w, mm.tokens(cfg, 9), [9])


def test_slow_decay_keeps_the_first_token():
    """decays near one and small steps: what the first token wrote is still read hundreds of tokens later"""
    cfg = mm.config([mm.delta(2, 1, 32, 32)], width=64, vocab=64)
    w = mm.weights(cfg, 12)
    w["l0.mix.A_log"][:] = -6.0
    w["l0.mix.dt_bias"][:] = -4.0
    toks = mm.tokens(cfg, 400)
    other = [toks[0] ^ 1] + toks[1:]
    a, b = mixers.zuselix(cfg, w, toks)[0], mixers.zuselix(cfg, w, other)[0]
    assert error(a[300:], b[300:]) > 1e-3  # (the first token shows)
    for cuts in ([400], [130, 200, 1, 69], [64] * 6 + [16], [397, 1, 1, 1]):
        check(cfg, w, toks, cuts, max_seq=400, tol=5e-5)


def test_large_decays_and_steps():
    """decays that forget everything at once, and keys that repeat with steps near one"""
    cfg = mm.config([mm.delta(4, 2, 16, 16)], width=64, vocab=8)
    for a_log, dt in ((3.0, 3.0), (-8.0, -8.0), (1.0, 8.0)):
        w = mm.weights(cfg, 13, b=6.0)
        w["l0.mix.A_log"][:] = a_log
        w["l0.mix.dt_bias"][:] = dt
        check(cfg, w, mm.tokens(cfg, 150), [140] + [1] * 10, tol=1e-4)


def test_long_decoding():
    cfg = mm.config([mm.delta(2, 1, 16, 32), mm.latent(2, 16, 16, 32, 0.3, 48)], width=64, vocab=100)
    check(cfg, mm.weights(cfg, 14), mm.tokens(cfg, 700), [4] + [1] * 696, max_seq=700, tol=5e-5)


def oracle_greedy(cfg, w, prompt, steps):
    toks, margin = list(prompt), []
    for _ in range(steps):
        logits = mixers.zuselix(cfg, w, toks)[0][-1]
        top = np.sort(logits)
        margin.append(top[-1] - top[-2])
        toks.append(int(np.argmax(logits)))
    return toks[len(prompt):], min(margin)


@pytest.mark.parametrize("graph", [1, 0])
@pytest.mark.parametrize("plen", [3, 20])
def test_greedy_generation(plen, graph):
    """through the framework's loop: on the device and token by token over the host"""
    from caten_amd import _lib, llm
    cfg = MODELS["stack"]
    w = mm.weights(cfg, 15)
    prompt = mm.tokens(cfg, plen, 3)
    want, margin = oracle_greedy(cfg, w, prompt, 30)
    assert margin > 1e-3
    lib = _lib.init()
    _lib.check(lib.cthip_set_option(b"decoder_graph", graph))
    try:
        m = mm.session(cfg, w)
        for _ in range(3):  # captured graphs replay on a session that has run
            assert llm.gpt2_generate(m, prompt, 30, on_device=True) == want
        assert llm.gpt2_generate(m, prompt, 30, on_device=False) == want
        m.close()
    finally:
        _lib.check(lib.cthip_set_option(b"decoder_graph", 1))


def test_generation_stops_and_goes_on():
    """steps queued behind the end token leave the recurrent state as it is: the sequence continues as if they had not run"""
    cfg = MODELS["stack"]
    w = mm.weights(cfg, 16)
    prompt = mm.tokens(cfg, 12, 4)
    free, _ = oracle_greedy(cfg, w, prompt, 24)
    k = next(i for i in range(2, 24) if free[i] not in free[:i])
    m = mm.session(cfg, w)
    first = m.forward(prompt, len(prompt), 0)
    got = m.generate_until(200, free[k])
    assert [first] + got == free[:k + 1]
    assert m.position == len(prompt) + len(got)
    toks = prompt + free[:k + 1] + mm.tokens(cfg, 5, 5)
    rest = toks[m.position:]
    logits = m.forward_rows(rest, range(len(rest)), m.position)[1]
    assert error(logits, mixers.zuselix(cfg, w, toks)[0][-len(rest):]) < TOL["float32"]
    m.close()


def test_generate_in_pieces():
    cfg = MODELS["stack"]
    w = mm.weights(cfg, 19)
    prompt = mm.tokens(cfg, 10, 6)
    want, margin = oracle_greedy(cfg, w, prompt, 40)
    assert margin > 1e-3
    m = mm.session(cfg, w)
    out = [m.forward(prompt, len(prompt), 0)]
    for k in (1, 8, 3, 17, 10):
        out += m.generate_on_device(k)
    assert out == want
    m.close()


def test_state_and_cache_against_the_equations():
    """the recurrent matrices and the cached latents themselves, after a prompt and decoded tokens"""
    cfg = mm.config([mm.delta(4, 2, 24, 40, 4), mm.latent(3, 16, 16, 40, 0.3)], width=96)
    w = {k: v.astype(np.float64) for k, v in mm.weights(cfg, 18).items()}
    toks = mm.tokens(cfg, 50)
    m = mm.session(cfg, mm.weights(cfg, 18), max_seq=64)
    all_rows(m, toks, [45, 1, 1, 3])
    x = w["embed"][toks] + mixers.sinusoid(range(50), 96)
    h = mixers.layer_norm(x, w["l0.norm1"], 1e-5)
    k = mixers.unit(mixers.short_conv(h @ w["l0.mix.k"].T, w["l0.mix.k.conv"]).reshape(50, 2, 24))
    v = mixers.short_conv(h @ w["l0.mix.v"].T, w["l0.mix.v.conv"]).reshape(50, 4, 40)
    beta = mixers.sigmoid(h @ w["l0.mix.b"].T)
    g = np.exp(-np.exp(w["l0.mix.A_log"]) * mixers.softplus(h @ w["l0.mix.a"].T + w["l0.mix.dt_bias"]))
    S = m.peek("state.0").reshape(4, 48, 32)
    for n in range(4):
        _, want = mixers.delta_recurrence(k[:, n // 2], k[:, n // 2], v[:, n], g[:, n], beta[:, n])
        np.testing.assert_allclose(S[n, :40, :24], want.T, rtol=0, atol=2e-6 * np.abs(want).max() + 1e-6)
        assert not S[n, 40:].any() and not S[n, :, 24:].any()
    x = x + mixers.delta_mixer(h, cfg["layers"][0]["mixer"], lambda s: w["l0.mix." + s], 1e-5)
    c = mixers.rms_norm(mixers.layer_norm(x, w["l1.norm1"], 1e-5) @ w["l1.mix.dkv"].T, w["l1.mix.dkv.norm"], 1e-5)
    cache = m.peek("latent.1").reshape(64, 48)
    np.testing.assert_allclose(cache[:50, :40], c, rtol=0, atol=3e-5)
    assert not cache[:, 40:].any()
    m.close()


def test_model_directory_and_trace_replay(tmp_path):
    """a directory as a user has it, through load_model and the replay program"""
    import importlib.machinery
    import importlib.util
    import json
    import os
    from caten_amd import llm, safetensors
    cfg = MODELS["stack"]
    w = mm.weights(cfg, 19)
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    safetensors.write(str(tmp_path / "model.safetensors"), mm.raw_tensors(w))
    path = os.path.join(os.path.dirname(os.path.dirname(os.path.abspath(__file__))), "bin", "trace_run")
    loader = importlib.machinery.SourceFileLoader("trace_run", path)
    mod = importlib.util.module_from_spec(importlib.util.spec_from_loader("trace_run", loader))
    loader.exec_module(mod)
    a, b = mm.tokens(cfg, 60, 7), mm.tokens(cfg, 9, 8)
    want = {"a": mixers.zuselix(cfg, w, a)[0], "b": mixers.zuselix(cfg, w, b)[0]}
    for dtype in ("float32", "bfloat16"):
        r = mod.Replay(llm.load_model(str(tmp_path), dtype, max_seq=60), str(tmp_path))
        steps = [("a", a[:50], [49, 3, 3], 0, False), ("a", a[50:53], [0, 2], 50, False), ("a", a[53:], [], 53, True), ("b", b, [0, 8], 0, True)]
        for i, (rid, toks, rows, at, end) in enumerate(steps):
            r.step({"step": i, "entries": [{"id": rid, "tokens": toks, "want": rows}], "end": [rid] if end else []})
            out = tmp_path / f"{i}.f32"
            assert out.exists() == bool(rows)
            if rows:
                got = np.fromfile(out, "<f4").reshape(len(rows), -1)
                assert error(got, want[rid][[at + k for k in rows]]) < TOL[dtype]
                out.unlink()
        with pytest.raises(ValueError, match="one sequence"):
            r.step({"step": 9, "entries": [{"id": "x", "tokens": [1], "want": []}, {"id": "y", "tokens": [1], "want": []}], "end": []})
        r.model.close()


def test_rows_of_the_other_models():
    """forward_rows on GPT-2 and Llama shaped sessions: the logits a forward of every prefix ends with"""
    from caten_amd import llm, synth
    for make, sd, cfg in ((llm.make_gpt2, llm.gpt2_state_dict(synth.gpt2_weights(synth.GPT2_CONFIGS["gpt2-tiny"]), "q8_0"), synth.GPT2_CONFIGS["gpt2-tiny"]),
                          (llm.make_llama, llm.llama_state_dict(synth.llama_weights(synth.LLAMA_CONFIGS["llama-tiny"]), "bf16"), synth.LLAMA_CONFIGS["llama-tiny"])):
        m = make(cfg, sd)
        toks = synth.prompt(cfg["vocab"], 20, 3)
        for n in (5, 20):
            rows = [0, n - 2, n - 1]
            got = m.forward_rows(toks[:n], rows, 0)[1]
            for r, row in zip(rows, got):
                _, want = m.forward(toks[:r + 1], r + 1, 0, return_logits=True)
                np.testing.assert_allclose(row, want, rtol=1e-3, atol=1e-4)
        m.close()


@pytest.mark.parametrize("cols", [8, 120, 128, 768, 1000, 2048, 6144, 8192])
def test_bf16_linear(cols):
    """bf16 weights: one row and several through every kernel family, against the same values in float64"""
    from caten_amd import _lib, ops
    from caten_amd.quant import from_bf16, to_bf16
    lib = _lib.init()
    rng = np.random.default_rng(cols)
    rows = 130
    bits = to_bf16(rng.standard_normal(rows * cols).astype(np.float32))
    W = from_bf16(bits).reshape(rows, cols)
    h = ops.WeightMatrix("bf16", bits.view(np.uint8), rows, cols)
    assert np.array_equal(h.dequantize(), W)
    assert np.array_equal(ops.dequantize("bf16", bits.view(np.uint8), 100), W.ravel()[:100])
    for m in (1, 3, 40):
        x = rng.standard_normal((m, cols)).astype(np.float32)
        want = x.astype(np.float64) @ W.T.astype(np.float64)
        for prec, tol in ((0, 1e-5), (3, 1e-5), (2, 1e-4), (1, 2e-2)):
            _lib.check(lib.cthip_set_option(b"gemm_precision", prec))
            try:
                got = ops.linear(x, h)
            finally:
                _lib.check(lib.cthip_set_option(b"gemm_precision", 2))
            assert np.abs(got - want).max() / np.sqrt((want ** 2).mean()) < tol, (m, prec)
    h.free()


def test_what_a_mixed_decoder_refuses():
    from caten_amd import _lib, llm
    from caten_amd._lib import HipError
    cfg = MODELS["latent"]
    w = mm.weights(cfg, 20)
    for layer, msg in ((mm.delta(dim=264), "at most 256"), (mm.delta(3, 2), "bad argument"), (mm.latent(kv_rank=1040), "at most 1024"),
                       (mm.delta(conv=0), "bad argument")):
        with pytest.raises(HipError, match=msg):
            mm.session(mm.config([layer]), {})
    short = dict(w)
    del short["l0.mix.uk"]
    with pytest.raises(HipError, match="1 tensors of the model are missing"):
        mm.session(cfg, short)
    with pytest.raises(HipError, match="not a tensor of this model"):
        mm.session(cfg, dict(w, extra=w["embed"]))
    m = mm.session(cfg, dict(w, **{"l0.mix.uk": w["l0.mix.uk"][:, :40]}))
    with pytest.raises(HipError, match="l0.mix.uk.*expected"):
        m.forward([1], 1, 0)
    m.close()
    sd = llm.safetensors_state_dict(mm.raw_tensors(w))
    sd["l0.mix.dkv"] = llm.Tensor.from_f32(w["l0.mix.dkv"], "f32")
    m = llm.MixedTransformer(dict(llm.zuselix_config(cfg), max_seq=16)).load_state_dict(sd)
    with pytest.raises(HipError, match="its neighbours"):
        m.forward([1], 1, 0)
    m.close()
    lib = _lib.init()
    _lib.check(lib.cthip_set_option(b"kv_cache", 1))
    try:
        m = mm.session(cfg, w)
        with pytest.raises(HipError, match="fp32 rows"):
            m.forward([1], 1, 0)
        m.close()
    finally:
        _lib.check(lib.cthip_set_option(b"kv_cache", 0))
