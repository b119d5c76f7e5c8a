"""Matalix models (sliding-window attention beside lightning attention, looped layers) against the plain float64 restatement
in oracle/mixers.py."""
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
