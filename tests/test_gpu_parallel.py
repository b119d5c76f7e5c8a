"""Matalix models (sliding-window attention beside lightning attention, looped layers) and their mixers one by one, against
the plain float64 restatement in oracle/mixers.py."""
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


def check(cfg, w, toks, cuts, dtype="float32", max_seq=256, tol=None, want=None):
    want = mixers.matalix(cfg, w, toks)[0] if want is None else want
    m = mm.session(cfg, w, dtype, max_seq)
    got = all_rows(m, toks, cuts)
    m.close()
    e = error(got, want)
    assert e < (tol or TOL[dtype]), (e, np.abs(got - want).max(1) / np.sqrt((want ** 2).mean()))


MODELS = {
    "one": mm.matalix([mm.parallel()]),
    "one_mlp": mm.matalix([mm.parallel(ff=192)]),
    "stack": mm.matalix([mm.parallel(ff=96), mm.parallel(mm.window(6, 2, 48, 16, 33)), mm.parallel(mm.window(2, 2), ff=224)]),
    "loop": mm.matalix([mm.parallel(ff=64), mm.parallel(), mm.parallel(ff=64, limit=0.5)], loop=dict(start=1, stop=3, times=3)),
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
    check(cfg, mm.weights(cfg, 2), mm.tokens(cfg, 60), [1] * 60, dtype)


# sizes that are multiples of nothing; one head and many; every sharing of key heads from none to seven queries; values wider
# and narrower than keys; rotations of a part of a head; layers of one model that differ in everything
W, N, P = mm.window, mm.lightning, mm.parallel
ODD = {
    "one_head_each": mm.matalix([P(W(1, 1, 12, 7, 5, dims=6), N(1, 8, 5), ff=50)], width=64, vocab=33),
    "unshared": mm.matalix([P(W(3, 3, 24, 40, 9, dims=20), N(3, 24, 40), ff=88)], width=96, vocab=301),
    "three_to_one": mm.matalix([P(W(3, 1, 20, 20, 17), N(5, 40, 24))], width=80),
    "five_to_one": mm.matalix([P(W(10, 2, 16, 16, 12, dims=2), N(2, 16, 80), ff=36)], width=176),
    "seven_to_one": mm.matalix([P(W(7, 1, 32, 8, 30), N(7, 8, 8))], width=64),
    "eight_to_one": mm.matalix([P(W(16, 2, 16, 16, 64), N(20, 16, 16), ff=64)], width=160),
    "wide_heads": mm.matalix([P(W(2, 1, 256, 256, 20, scale=0.06), N(2, 256, 256))], width=256),
    "wide_shared": mm.matalix([P(W(6, 1, 192, 136, 20, scale=0.07), N(1, 136, 200))], width=128),
    "wide_state_narrow_heads": mm.matalix([P(W(8, 2, 16, 16, 20), N(2, 200, 16))], width=128),
    "wide_values": mm.matalix([P(W(4, 2, 16, 160, 20), N(3, 16, 144))], width=128),
    "one_token_window": mm.matalix([P(W(size=1), ff=32), P(W(size=2))]),
    "window_beyond_the_sequence": mm.matalix([P(W(size=5000))]),
    "different_layers": mm.matalix([P(W(2, 1, 40, 24, 7, 0.3, 16), N(4, 12, 20), 1.0, 1.0, 72, 0.3), P(W(6, 3, 8, 48, 50, 0.5), N(1, 64, 64), 0.2, 3.0),
                                    P(W(5, 5, 28, 28, 16, 0.1, base=500.0, factor=1.0), N(6, 20, 8), -0.5, 0.5, 40, 50.0)], width=112, eps=0.03),
    "width_not_16": mm.matalix([P(W(2, 1, 16, 16), N(2, 16, 16), ff=72), P(ff=36)], width=104),
    "width_not_8": mm.matalix([P(W(2, 1, 16, 16), N(2, 16, 16), ff=30), P(ff=27)], width=90),
    "width_odd": mm.matalix([P(W(2, 1, 16, 16), N(2, 16, 16), ff=31)], width=77, vocab=65),
}


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", list(ODD))
def test_sizes(name, dtype):
    """a prompt, portions and single tokens, on sizes that exercise padding and every fallback"""
    cfg = ODD[name]
    check(cfg, mm.weights(cfg, 3), mm.tokens(cfg, 60), [33, 2, 9, 1, 1, 14], dtype)


@pytest.mark.parametrize("cuts", [[100], [2] * 50, [3] * 33 + [1], [7] * 14 + [2], [8] * 12 + [4], [31, 32, 33, 4], [1, 64, 35], [65, 35],
                                  [15, 16, 17, 52], [23, 24, 25, 28], [63, 1, 36]])
@pytest.mark.parametrize("name", ["stack", "loop"])
def test_portions(name, cuts):
    """however the tokens are cut, the logits are those of the whole sequence"""
    cfg = MODELS[name]
    check(cfg, mm.weights(cfg, 4), mm.tokens(cfg, 100), cuts)


@pytest.mark.parametrize("loop", [None, dict(start=0, stop=1, times=1), dict(start=0, stop=1, times=4), dict(start=2, stop=3, times=2),
                                  dict(start=0, stop=3, times=2), dict(start=1, stop=2, times=3)])
def test_loops(loop):
    """passes at the front, in the middle, at the end, over everything; each keeps its own keys, values and state"""
    cfg = mm.matalix([P(ff=48), P(W(2, 2, 16, 16, 9)), P(right=N(2, 24, 8), ff=40)])
    cfg["loop"] = loop
    w = mm.weights(cfg, 5)
    toks = mm.tokens(cfg, 50)
    for cuts in ([50], [30, 2, 1, 1, 16], [1] * 50):
        check(cfg, w, toks, cuts)


def test_the_embedding_enters_every_pass():
    """left out of a pass it shows, and so does one key cache for all passes"""
    cfg = mm.matalix([P(ff=48), P()], loop=dict(start=0, stop=2, times=3))
    w, toks = mm.weights(cfg, 5), mm.tokens(cfg, 40)
    once = dict(cfg, layers=cfg["layers"] * 3, loop=None)
    flat = dict(w, **{f"l{i}.{k[3:]}": v for i in range(2, 6) for k, v in w.items() if k.startswith(f"l{i % 2}.")})
    want = mixers.matalix(cfg, w, toks)[0]
    assert error(mixers.matalix(once, flat, toks)[0], want) > 0.1
    check(cfg, w, toks, [25] + [1] * 15, want=want)


def test_sequences_one_after_another():
    """a sequence that starts at position 0 sees nothing of the ones before it, whatever their length"""
    cfg = MODELS["loop"]
    w = mm.weights(cfg, 6)
    m = mm.session(cfg, w)
    for seed, cuts in enumerate([[90], [1, 1, 1], [20, 1, 1], [2], [50, 2, 9], [1] * 12, [8], [1] * 30, [200], [30]]):
        toks = mm.tokens(cfg, sum(cuts), seed)
        assert error(all_rows(m, toks, cuts), mixers.matalix(cfg, w, toks)[0]) < TOL["float32"], seed
    m.close()


def test_rows_left_by_another_sequence_need_not_be_numbers():
    """rings and states that hold NaN where no token of this sequence has written"""
    from caten_amd import _lib
    import ctypes as C
    cfg = mm.matalix([P(W(size=200))])
    w = mm.weights(cfg, 6)
    m = mm.session(cfg, w)
    m.forward_rows([1], [], 0)
    bad = np.full(200 * 2 * 32, np.nan, np.float32)
    for what in ("keys.0", "values.0", "state.0"):
        p, n = C.c_void_p(), C.c_int64()
        _lib.check(m.lib.cthip_decoder_peek(m.handle, what.encode(), C.byref(p), C.byref(n)))
        assert n.value <= bad.size
        _lib.check(m.lib.cthip_h2d(p.value, bad.ctypes.data, 4 * n.value))
    for cuts in ([1] * 30, [20, 1, 1]):
        toks = mm.tokens(cfg, sum(cuts), 1)
        assert error(all_rows(m, toks, cuts), mixers.matalix(cfg, w, toks)[0]) < TOL["float32"]
    m.close()


def test_state_does_not_go_back():
    cfg = MODELS["one"]
    m = mm.session(cfg, mm.weights(cfg, 6))
    from caten_amd._lib import HipError
    m.forward_rows(list(range(12)), [], 0)
    for n in (11, 13):
        with pytest.raises(HipError, match="starts there or at 0"):
            m.forward_rows([1], [0], n)
    m.forward_rows([1], [0], 12)
    m.close()


# ---- keys that stand out, at the window's edges ----
def asking_model(size, heads=4, kv_heads=2, dims=16):
    """token 1 asks for token 2: in the unrotated half of a head its query meets that token's key, whatever lies between"""
    cfg = mm.matalix([P(W(heads, kv_heads, 32, 16, size, 0.5, dims), N(1, 16, 16), 1.5, 0.05)], width=96, vocab=200)
    w = mm.weights(cfg, 8)
    rng = np.random.default_rng(9)
    signs = rng.choice([-1.0, 1.0], (2, 96)).astype(np.float32)
    basis = np.linalg.qr(signs.T)[0]
    w["embed"] -= w["embed"] @ basis @ basis.T  # (no other token asks or answers)
    w["embed"][1], w["embed"][2] = 2 * signs[0], 2 * signs[1]
    w["l0.norm1"][:] = 0
    rms = [np.sqrt((e ** 2).mean()) for e in w["embed"][1:3]]
    head = np.zeros(32, np.float32)
    head[dims:] = rng.choice([-1.0, 1.0], 32 - dims)
    for name, e, r, n in (("q", w["embed"][1], rms[0], heads), ("k", w["embed"][2], rms[1], kv_heads)):
        w[f"l0.mix.left.{name}"] = 0.2 * w[f"l0.mix.left.{name}"] + np.tile(np.outer(head, e / r) / 96 * 8, (n, 1))
        w[f"l0.mix.left.{name}.b"] *= 0.1
        w[f"l0.mix.left.{name}.norm"][:] = 1.0
    w["l0.mix.left.o"] *= 6
    return cfg, {k: mm.as_bf16(v) for k, v in w.items()}


@pytest.mark.parametrize("size", [2, 16, 17, 31, 32, 33, 63, 64, 65, 100, 256, 300, 520])
def test_window_edges(size):
    """a key that carries the softmax, exactly at the window's far end and one past it: asked for in a prompt, in a later
    portion and by decoded tokens; in the oracle a window off by one shows"""
    cfg, w = asking_model(size)
    T = size + 90
    toks = [3 + t % 190 for t in mm.tokens(cfg, T)]
    key = [5, 50]
    for at in key:
        toks[at] = 2
    asks = [at + size - 1 for at in key] + [at + size for at in key]
    for t in asks:
        toks[t] = 1
    want = mixers.matalix(cfg, w, toks)[0]
    scale = np.sqrt((want ** 2).mean())
    for d in (-1, 1):
        off = dict(cfg, layers=[dict(cfg["layers"][0], mixer=dict(cfg["layers"][0]["mixer"], left=dict(cfg["layers"][0]["mixer"]["left"], mask={"size": size + d})))])
        shows = np.abs(mixers.matalix(off, w, toks)[0] - want).max(1) / scale
        assert shows[asks[1 if d < 0 else 3]] > 0.3, d
    for dtype in ("float32", "bfloat16"):
        for cuts in ([T], [size + 2, T - size - 2], [size - 1] + [1] * (T - size + 1)):
            check(cfg, w, toks, cuts, dtype, T, want=want)


@pytest.mark.parametrize("at", [0, 1, 15, 16, 31, 32, 63, 64, 255, 511, 512])
def test_far_key(at):
    """one key among hundreds carries the softmax: at borders of tiles and key ranges, at the first position"""
    cfg, w = asking_model(600)
    toks = [3 + t % 190 for t in mm.tokens(cfg, 560)]
    toks[at] = 2
    toks[530] = toks[540] = toks[559] = 1
    want = mixers.matalix(cfg, w, toks)[0]
    without = list(toks)
    without[at] = 7
    blind = mixers.matalix(cfg, w, without)[0]
    assert np.abs(want[559] - blind[559]).max() / np.sqrt((want ** 2).mean()) > 0.3  # (the key shows in the logits)
    for dtype in ("float32", "bfloat16"):
        check(cfg, w, toks, [535, 20] + [1] * 5, dtype, 576, want=want)


@pytest.mark.parametrize("n", [1, 2, 15, 16, 17, 63, 64, 65, 127, 128, 129, 255, 256, 257, 999, 1000, 1001, 1063, 1100])
def test_decode_at_tile_and_range_borders(n):
    """the first decoded tokens behind prompts that end around the borders of key tiles, key ranges and the ring"""
    cfg = mm.matalix([P(W(3, 1, 16, 16, 1000, 0.3), N(2, 16, 16)), P(W(4, 4, 16, 16, 70, 0.3), N(1, 16, 16))], width=64, vocab=100)
    check(cfg, mm.weights(cfg, 10), mm.tokens(cfg, n + 3), [n, 1, 1, 1], max_seq=1200)


def test_long_windows_in_decode():
    """more rows than the key ranges take in one round; a ring whose length is no multiple of a tile"""
    cfg = mm.matalix([P(W(40, 20, 16, 16, 2999, 0.3), N(1, 16, 16))], width=64, vocab=100)
    w, toks = mm.weights(cfg, 10), mm.tokens(cfg, 3205)
    want = mixers.matalix(cfg, w, toks)[0]
    check(cfg, w, toks, [2990, 1, 1, 203] + [1] * 10, max_seq=3300, want=want)


# ---- rotation ----
@pytest.mark.parametrize("dims,base,factor,original,fast,slow", [
    (32, 10000.0, 4.0, 64, 8.0, 1.0), (32, 10000.0, 16.0, 4096, 32.0, 1.0), (20, 500.0, 2.0, 16, 4.0, 2.0), (2, 100.0, 3.0, 100, 2.0, 1.0),
    (32, 1e6, 1.0, 64, 32.0, 1.0), (16, 50.0, 40.0, 8, 1.0, 1.0), (32, 10000.0, None, None, None, None), (8, 7.0, 2.5, 3, 30.0, 0.1)])
def test_rotations(dims, base, factor, original, fast, slow):
    """ramps of every shape (wide, of no width, clipped at either end), without scaling, over a part of a head; positions of
    thousands keep their angles"""
    left = W(2, 1, 32, 16, 1500, 1.5, dims, base)
    left["rot"]["scaling"] = None if factor is None else dict(factor=factor, original=original, fast=fast, slow=slow)
    cfg = mm.matalix([P(left, N(1, 16, 16), 1.5, 0.1)], width=64, vocab=100)
    w, toks = mm.weights(cfg, 11), mm.tokens(cfg, 1400)
    check(cfg, w, toks, [1380, 9] + [1] * 11, max_seq=1400, tol=1e-4)


# ---- the sink and the first tokens ----
def test_first_tokens_and_the_sink():
    """with few visible keys the sink takes its share; scores far below it, around it, far above it"""
    cfg = mm.matalix([P(W(size=4), left_scale=2.0)])
    w = mm.weights(cfg, 11)
    toks = mm.tokens(cfg, 11)
    for norm in (0.05, 1.0, 4.0):
        v = dict(w, **{"l0.mix.left.q.norm": mm.as_bf16(norm * w["l0.mix.left.q.norm"]), "l0.mix.left.k.norm": mm.as_bf16(norm * w["l0.mix.left.k.norm"])})
        want = mixers.matalix(cfg, v, toks)[0]
        for cuts in ([1] * 11, [11], [2, 9]):
            check(cfg, v, toks, cuts, tol=5e-5, want=want)
    blind = np.array([mixers.sink_softmax(np.zeros((1, 1)), s)[0, 0] for s in (-np.inf, 0.0)])
    assert np.array_equal(blind, [1.0, 0.5])


# ---- lightning attention ----
@pytest.mark.parametrize("decay", [[0.0, 1.0, 0.5], [0.9999, 0.99999, 1e-6], [0.95, 0.3, 0.999]])
@pytest.mark.parametrize("cuts", [[300], [63, 1, 64, 65, 107], [290] + [1] * 10, [2] * 150, [9, 64, 128, 99]])
def test_decays(decay, cuts):
    """decays from nothing to everything, portions on and off the chunks' borders"""
    cfg = mm.matalix([P(W(size=3), N(3, 16, 32, decay), 0.1, 1.5)], width=64, vocab=64)
    w, toks = mm.weights(cfg, 12), mm.tokens(cfg, 300)
    want = mixers.matalix(cfg, w, toks)[0]
    other = [toks[0] ^ 1] + toks[1:]
    if min(1 - d for d in decay) < 1e-4:  # (the first token shows at the end)
        assert error(mixers.matalix(cfg, w, other)[0][290:], want[290:]) > 1e-4
    check(cfg, w, toks, cuts, max_seq=300, tol=5e-5, want=want)


def test_prompt_of_more_chunks_than_are_held_at_once():
    cfg = mm.matalix([P(W(1, 1, 16, 16, 10), N(1, 16, 16, [0.9995]), 0.2, 1.0)], width=64, vocab=64)
    check(cfg, mm.weights(cfg, 13), mm.tokens(cfg, 4300), [4290, 1, 9], max_seq=4300, tol=1e-4)


def test_long_decoding():
    cfg = mm.matalix([P(W(2, 1, 16, 16, 50, 0.3), N(2, 16, 32, [0.998, 0.8]), ff=48), P(W(2, 2, 16, 16, 300), N(1, 16, 16, [0.9]))], width=64, vocab=100)
    check(cfg, mm.weights(cfg, 14), mm.tokens(cfg, 700), [4] + [1] * 696, max_seq=700, tol=5e-5)


# ---- the gated unit ----
@pytest.mark.parametrize("limit", [0.05, 0.7, 3.0, 1e4])
def test_clamps(limit):
    """gate clamped from above only, up from both sides; one row and several"""
    cfg = mm.matalix([P(ff=96, limit=limit)])
    w = mm.weights(cfg, 15, gate=3.0, up=3.0)
    toks = mm.tokens(cfg, 40)
    for dtype in ("float32", "bfloat16"):
        for cuts in ([40], [1] * 40):
            check(cfg, w, toks, cuts, dtype)


# ---- one mixer per layer, each option by itself ----
SINGLE = {
    "window_plain": dict(mixer="window"),
    "window_bias": dict(mixer="window", bias=True),
    "window_norm": dict(mixer="window", qk_norm=True),
    "window_gate": dict(mixer="window", gate=True),
    "window_rot": dict(mixer="window", rot=dict(dims=12, base=300.0)),
    "window_sink": dict(mixer="window", sink="tensor"),
    "window_zero_sink": dict(mixer="window", sink="zero"),
    "window_everything": dict(mixer="window", bias=True, qk_norm=True, gate=True, sink="tensor", out_scale=-1.7, rot=dict(dims=16, base=300.0, factor=4.0, original=32, fast=4.0, slow=1.0)),
    "lightning": dict(mixer="lightning"),
    "lightning_scale": dict(mixer="lightning", out_scale=0.3),
}


@pytest.mark.parametrize("name", list(SINGLE))
def test_single_mixers(name):
    """layers of one mixer without its usual company: plain norms, a head of its own, SwiGLU, no layer scale"""
    from caten_amd import llm
    opt, D, V, eps, T = SINGLE[name], 64, 90, 1e-5, 60
    window = opt["mixer"] == "window"
    m = dict(W(4, 2, 16, 24, 19, 0.3), rot=None) if window else N(3, 16, 24, [0.9, 0.5, 0.99])
    rng = np.random.default_rng(16)
    shapes = {"q": (64 if window else 48, D), "k": (32 if window else 48, D), "v": (48 if window else 72, D), "o": (D, 96 if window else 72)}
    if not window or opt.get("gate"):
        shapes["g"] = (96 if window else 72, D)
    if not window:
        shapes["norm"] = (72,)
    if opt.get("bias"):
        shapes.update({"q.b": (64,), "k.b": (32,), "v.b": (48,)})
    if opt.get("qk_norm"):
        shapes.update({"q.norm": (64,), "k.norm": (32,)})
    if opt.get("sink") == "tensor":
        shapes["sink"] = (4,)
    w = {"embed": (V, D), "head": (V, D), "final.norm": (D,), "l0.norm1": (D,), "l0.norm2": (D,), "l0.mlp.gate": (40, D), "l0.mlp.up": (40, D),
         "l0.mlp.down": (D, 40), **{"l0.mix." + k: s for k, s in shapes.items()}}
    w = {k: mm.as_bf16(rng.standard_normal(s) / (np.sqrt(s[-1]) if len(s) == 2 and k != "embed" else 1.0)) for k, s in w.items()}
    cfg = dict(vocab=V, dim=D, max_seq=64, eps=eps, norm="rmsnorm", precision=0,
               layers=[dict({k: v for k, v in m.items() if k not in ("mask", "rot")}, ffn=40, **({"window": 19} if window else {}), **opt)])
    model = llm.MixedTransformer(cfg).load_state_dict(llm.safetensors_state_dict(mm.raw_tensors(w), widen=True))
    t = {k: v.astype(np.float64) for k, v in w.items()}
    toks = [int(x) for x in rng.integers(0, V, T)]
    x = t["embed"][toks]
    h = mixers.rms_norm(x, t["l0.norm1"], eps)

    def of(n):
        return t["l0.mix." + n]
    if window:
        rot = opt.get("rot")
        if rot:
            rest = {k: v for k, v in rot.items() if k not in ("dims", "base")}
            m["rot"] = dict(dims=rot["dims"], base=rot["base"], scaling=rest or None)
        sink = {None: -np.inf, "zero": 0.0}[opt.get("sink")] if opt.get("sink") != "tensor" else of("sink")
        y = mixers.window_attention(h, m, of, eps, bool(opt.get("bias")), bool(opt.get("qk_norm")), sink, bool(opt.get("gate")))
    else:
        y = mixers.lightning_attention(h, m, of, eps)
    x = x + opt.get("out_scale", 1.0) * y
    x = x + mixers.dense_mlp(mixers.rms_norm(x, t["l0.norm2"], eps), lambda n: t["l0.mlp." + n])
    want = mixers.rms_norm(x, t["final.norm"], eps) @ t["head"].T
    for cuts in ([T], [1] * T, [30, 2, 9, 1, 18]):
        assert error(all_rows(model, toks, cuts), want) < TOL["float32"], cuts
    model.close()


def test_two_of_a_kind_side_by_side():
    """two window mixers, two lightning mixers, and lightning on the left"""
    from caten_amd import llm
    for kinds in (("window", "window"), ("lightning", "lightning"), ("lightning", "window")):
        D, V, eps, T = 64, 70, 1e-5, 50
        rng = np.random.default_rng(17)
        w = {"embed": (V, D), "head": (V, D), "final.norm": (D,), "l0.norm1": (D,)}
        layers, ms = [], []
        for side, kind in zip(("left", "right"), kinds):
            p = f"l0.mix.{side}."
            if kind == "window":
                m = dict(W(4, 2, 16, 16, 11 if side == "left" else 26, 0.3), rot=None)
                w.update({p + "q": (64, D), p + "k": (32, D), p + "v": (32, D), p + "o": (D, 64)})
                layers.append(dict(mixer="window", heads=4, kv_heads=2, dim=16, vdim=16, scale=0.3, window=m["mask"]["size"]))
            else:
                m = N(2, 16, 32, [0.9, 0.6] if side == "left" else [0.99, 0.2])
                w.update({p + "q": (32, D), p + "k": (32, D), p + "v": (64, D), p + "g": (64, D), p + "norm": (64,), p + "o": (D, 64)})
                layers.append(dict(m, mixer="lightning"))
            ms.append(m)
        w = {k: mm.as_bf16(rng.standard_normal(s) / (np.sqrt(s[-1]) if len(s) == 2 and k != "embed" else 1.0)) for k, s in w.items()}
        model = llm.MixedTransformer(dict(vocab=V, dim=D, max_seq=64, eps=eps, norm="rmsnorm", precision=0, layers=[dict(mixers=layers)]))
        model.load_state_dict(llm.safetensors_state_dict(mm.raw_tensors(w), widen=True))
        t = {k: v.astype(np.float64) for k, v in w.items()}
        toks = [int(x) for x in rng.integers(0, V, T)]
        x = t["embed"][toks]
        h = mixers.rms_norm(x, t["l0.norm1"], eps)
        for side, kind, m in zip(("left", "right"), kinds, ms):
            def of(n):
                return t[f"l0.mix.{side}.{n}"]
            x = x + (mixers.window_attention(h, m, of, eps, False, False, -np.inf, False) if kind == "window" else mixers.lightning_attention(h, m, of, eps))
        want = mixers.rms_norm(x, t["final.norm"], eps) @ t["head"].T
        for cuts in ([T], [1] * T, [30, 2, 9, 1, 8]):
            assert error(all_rows(model, toks, cuts), want) < TOL["float32"], (kinds, cuts)
        model.close()


# ---- the framework's loop ----
def generating(cfg, seed):
    """a small embedding and large mixers: with a tied head the likeliest next token would be the current one"""
    w = mm.weights(cfg, seed, ls1=4.0, ls2=4.0)
    w["embed"] = mm.as_bf16(w["embed"] / 4)
    return w


def oracle_greedy(cfg, w, prompt, steps):
    toks, margin = list(prompt), []
    for _ in range(steps):
        logits = mixers.matalix(cfg, w, toks)[0][-1]
        top = np.sort(logits)
        margin.append(top[-1] - top[-2])
        toks.append(int(np.argmax(logits)))
    return toks[len(prompt):], min(margin)


@pytest.mark.parametrize("graph", [1, 0])
@pytest.mark.parametrize("plen", [3, 20])
def test_greedy_generation(plen, graph):
    """through the framework's loop: on the device and token by token over the host"""
    from caten_amd import _lib, llm
    cfg = MODELS["loop"]
    w = generating(cfg, 18)
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
    """steps queued behind the end token change nothing that the sequence still reads, also where its rings have wrapped"""
    cfg = MODELS["loop"]
    w = generating(cfg, 19)
    prompt = mm.tokens(cfg, 40, 4)
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
    assert error(logits, mixers.matalix(cfg, w, toks)[0][-len(rest):]) < TOL["float32"]
    m.close()


def test_generate_in_pieces():
    cfg = MODELS["stack"]
    w = generating(cfg, 20)
    prompt = mm.tokens(cfg, 10, 6)
    want, margin = oracle_greedy(cfg, w, prompt, 40)
    assert margin > 1e-3
    m = mm.session(cfg, w)
    out = [m.forward(prompt, len(prompt), 0)]
    for k in (1, 8, 3, 17, 10):
        out += m.generate_on_device(k)
    assert out == want
    m.close()


def test_two_runs_are_bit_identical():
    cfg = MODELS["loop"]
    m = mm.session(cfg, mm.weights(cfg, 21), "bfloat16")
    toks = mm.tokens(cfg, 90)
    a, b = (all_rows(m, toks, [64, 2, 9] + [1] * 15) for _ in range(2))
    assert np.array_equal(a, b)
    m.close()


def test_state_and_rings_against_the_equations():
    """the recurrent matrices, keys and values themselves, after a prompt and decoded tokens, in every pass"""
    cfg = mm.matalix([P(W(4, 2, 24, 12, 20), N(2, 20, 40, [0.9, 0.99]))], width=96, loop=dict(start=0, stop=1, times=2))
    ws = mm.weights(cfg, 22)
    t = {k: v.astype(np.float64) for k, v in ws.items()}
    toks, T, eps = mm.tokens(cfg, 50), 50, 1e-5
    m = mm.session(cfg, ws, max_seq=64)
    all_rows(m, toks, [45, 1, 1, 3])
    x0 = x = t["embed"][toks]
    freqs, mscale = mixers.yarn(cfg["layers"][0]["mixer"]["left"]["rot"])
    for run in range(2):
        x = x + x0 if run else x
        h = mixers.rms_norm(x, 1 + t["l0.norm1"], eps)
        k = mixers.rms_norm(h @ t["l0.mix.left.k"].T + t["l0.mix.left.k.b"], t["l0.mix.left.k.norm"], eps).reshape(T, 2, 24)
        k = mixers.rotate_half(k, range(T), freqs, mscale)
        v = (h @ t["l0.mix.left.v"].T + t["l0.mix.left.v.b"]).reshape(T, 2, 12)
        K, V = m.peek(f"keys.{run}").reshape(20, 2, 32), m.peek(f"values.{run}").reshape(20, 2, 16)
        for p in range(30, 50):
            np.testing.assert_allclose(K[p % 20, :, :24], k[p], rtol=0, atol=3e-5)
            np.testing.assert_allclose(V[p % 20, :, :12], v[p], rtol=0, atol=3e-5)
        assert not K[:, :, 24:].any() and not V[:, :, 12:].any()
        kk, vv = (mixers.silu(h @ t["l0.mix.right." + n].T).reshape(T, 2, -1) for n in ("k", "v"))
        S = m.peek(f"state.{run}").reshape(2, 48, 32)
        for n in range(2):
            _, want = mixers.lightning_recurrence(kk[:, n], kk[:, n], vv[:, n], [0.9, 0.99][n])
            np.testing.assert_allclose(S[n, :40, :20], want.T, rtol=0, atol=3e-6 * np.abs(want).max())
            assert not S[n, 40:].any() and not S[n, :, 20:].any()
        x = x + t["l0.ls1"] * mixers.parallel_mixer(h, cfg["layers"][0]["mixer"], lambda n: t["l0.mix." + n], eps)
    m.close()


def test_model_directory_and_trace_replay(tmp_path):
    """a directory as a user has it, through load_model and the replay program"""
    import importlib.machinery
    import importlib.util
    import json
    import os
    from caten_amd import llm, safetensors
    cfg = MODELS["loop"]
    w = mm.weights(cfg, 23)
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    safetensors.write(str(tmp_path / "model.safetensors"), mm.raw_tensors(w))
    path = os.path.join(os.path.dirname(os.path.dirname(os.path.abspath(__file__))), "bin", "trace_run")
    loader = importlib.machinery.SourceFileLoader("trace_run", path)
    mod = importlib.util.module_from_spec(importlib.util.spec_from_loader("trace_run", loader))
    loader.exec_module(mod)
    a, b = mm.tokens(cfg, 60, 7), mm.tokens(cfg, 9, 8)
    want = {"a": mixers.matalix(cfg, w, a)[0], "b": mixers.matalix(cfg, w, b)[0]}
    for dtype in ("float32", "bfloat16"):
        r = mod.Replay(llm.load_model(str(tmp_path), dtype, max_seq=60), str(tmp_path))
        steps = [("a", a[:50], [49, 3, 3], 0, False), ("a", a[50:53], [0, 2], 50, False), ("a", a[53:], [6], 53, True), ("b", b, [0, 8], 0, True)]
        for i, (rid, toks, rows, at, end) in enumerate(steps):
            r.step({"step": i, "entries": [{"id": rid, "tokens": toks, "want": rows}], "end": [rid] if end else []})
            got = np.fromfile(tmp_path / f"{i}.f32", "<f4").reshape(len(rows), -1)
            assert error(got, want[rid][[at + k for k in rows]]) < TOL[dtype]
        r.model.close()


def test_what_is_refused():
    from caten_amd._lib import HipError
    for layer, msg in ((P(W(dim=264)), "at most 256"), (P(W(vdim=272)), "at most 256"), (P(right=N(dim=260)), "at most 256"), (P(W(3, 2)), "bad argument"),
                       (P(W(size=0)), "bad argument"), (P(W(dims=34)), "bad argument"), (P(W(dims=7)), "bad argument"),
                       (P(right=N(2, decay=[0.5, 1.5])), "bad argument")):
        with pytest.raises(HipError, match=msg):
            mm.session(mm.matalix([layer]), {})
    with pytest.raises(ValueError, match="2 decays for 3 heads"):
        mm.session(mm.matalix([P(right=N(3, decay=[0.5, 0.5]))]), {})
    for loop in (dict(start=1, stop=1, times=2), dict(start=0, stop=2, times=2), dict(start=-1, stop=1, times=2)):
        with pytest.raises(HipError, match="bad argument"):
            mm.session(mm.matalix([P()], loop=loop), {})
    cfg = MODELS["one"]
    w = mm.weights(cfg, 24)
    short = dict(w)
    del short["l0.mix.left.k.b"]
    with pytest.raises(HipError, match="1 tensors of the model are missing"):
        mm.session(cfg, short)
    with pytest.raises(HipError, match="not a tensor of this model"):
        mm.session(cfg, dict(w, head=w["embed"]))
    m = mm.session(cfg, dict(w, **{"l0.mix.right.norm": w["l0.mix.right.norm"][:-1]}))
    with pytest.raises(HipError, match="l0.mix.right.norm"):
        m.forward([1], 1, 0)
    m.close()
