"""Ranutar without a GPU: its configuration, and the plain statement (oracle/layered.py) against itself - portions and single tokens agree, every
mechanism matches a closed form where there is one, and mistakes planted in the oracle show at the inputs the GPU tests use."""
import copy

import numpy as np
import pytest

from oracle import layered as O
from tests import layered_util as U


def run(c, W, tokens, cuts=()):
    M = O.Model(c, W)
    s = O.Sequence(M)
    return np.concatenate([M.run(s, p) for p in np.split(np.asarray(tokens), list(cuts)) if len(p)])


def toks(c, n, seed=1):
    return np.random.default_rng(seed).integers(0, c["vocab"], n)


def test_oracle_does_not_depend_on_how_a_prompt_is_cut():
    c = U.sandwich_mixed()
    W, t = U.weights(c), toks(c, 50)
    whole = run(c, W, t)
    for cuts in ([1], [19], [2, 4, 6, 33], list(range(1, 50))):
        assert U.err(run(c, W, t, cuts), whole) < 1e-12


@pytest.mark.parametrize("moved", [-1, 1])
@pytest.mark.parametrize("window", [2, 16, 33, 64, 130])
def test_a_moved_window_shows_at_its_first_token(window, moved):
    c, edit = U.attracted(window)
    d = copy.deepcopy(c)
    d["layers"][0]["mixer"]["mask"]["size"] += moved
    W = U.weights(c)
    edit(W)
    for at in (0, 5):
        t = toks(c, at + window + 6)
        t[t == 7] = 8
        t[at] = 7
        a, b = run(c, W, t), run(d, W, t)
        first = at + window + min(moved, 0)   # the one position at which only one of the two sees the token
        assert U.err(a[first:first + 1], b[first:first + 1]) > 0.05


@pytest.mark.parametrize("kind,key", [("wkv", "S"), ("wkv", "h"), ("delta", "S"), ("delta", "q"), ("delta", "v"), ("conv1", "in"), ("conv2", "in")])
def test_a_lost_state_shows(kind, key):
    c = U.sandwich_mixed()
    M, t = O.Model(c, U.weights(c)), toks(c, 30)
    s, lost = O.Sequence(M), O.Sequence(M)
    M.run(s, t[:20])
    M.run(lost, t[:20])
    for st, L in zip(lost.state, c["layers"]):
        d = st.get(kind) if kind.startswith("conv") else st["mix"] if L["type"] == kind else None
        if d:
            d[key] = np.zeros_like(d[key])
    assert U.err(M.run(s, t[20:22]), M.run(lost, t[20:22])) > 0.02


def test_time_mixing_in_closed_form():
    """o_t = sum_{s<t} (r_t . k_s prod_{s<j<t} w_j) v_s + (r_t . u k_t) v_t"""
    rng = np.random.default_rng(0)
    n, d = 9, 5
    r, k, v = rng.normal(size=(3, n, d))
    w, u = rng.uniform(0.2, 1, (n, d)), rng.normal(size=d)
    S = np.zeros((d, d))
    for t in range(n):
        S, o = O.wkv_step(S, r[t], k[t], v[t], w[t], u)
        want = (r[t] * u * k[t]).sum() * v[t]
        for s in range(t):
            want = want + (r[t] * k[s] * w[s + 1:t].prod(0)).sum() * v[s]
        assert np.allclose(o, want)


def test_activation_meets_itself_at_zero():
    f = lambda z: O.xielu(np.array([z]), 0.3, -0.7)[0]
    assert f(0.0) == 0 and f(1e-6) == pytest.approx(5e-7, rel=1e-4) and f(-1e-6) == pytest.approx(-5e-7, rel=1e-4)
    assert f(2.0) == pytest.approx(np.log1p(np.exp(0.3)) * 4 + 1) and f(-30.0) == pytest.approx((0.5 + np.log1p(np.exp(-0.7))) * 29 - 15, rel=1e-6)


def test_rotation_keeps_the_rest_and_depends_on_distance_only():
    rot = {"base": 70.0, "dims": 6}
    q, k = np.random.default_rng(1).normal(size=(2, 8))
    a = O.rotate_halves(q, 11, rot)
    assert np.array_equal(a[6:], q[6:]) and np.linalg.norm(a) == pytest.approx(np.linalg.norm(q))
    assert a[0] == pytest.approx(q[0] * np.cos(11) - q[3] * np.sin(11)) and a[3] == pytest.approx(q[3] * np.cos(11) + q[0] * np.sin(11))
    assert a @ O.rotate_halves(k, 4, rot) == pytest.approx(O.rotate_halves(q, 107, rot) @ O.rotate_halves(k, 100, rot))


def test_convolution_sees_the_last_taps_only():
    w = np.random.default_rng(2).normal(size=(3, 4))
    h = np.zeros((9, 3))
    h[2] = [1, 2, 3]
    y = O.input_conv(h, w, {})
    assert np.allclose(y[2], h[2] * (1 + w[:, 3])) and np.allclose(y[5], h[2] * w[:, 0]) and not y[:2].any() and not y[6:].any()


def test_configuration_errors_name_the_key(tmp_path):
    import dsk
    good = U.sandwich_mixed()
    dsk.config_check(good)
    assert dsk.dir_architecture(U.save(tmp_path, good, {})) == "Ranutar"

    def broken(fn, match):
        c = copy.deepcopy(good)
        fn(c)
        with pytest.raises(dsk.DskError, match=match):
            dsk.config_check(c)
    broken(lambda c: c.pop("canon"), "canon")
    broken(lambda c: c["canon"].update(taps=0), "taps")
    broken(lambda c: c.pop("logit_scale"), "logit_scale")
    broken(lambda c: c["layers"][0].update(type="parallel"), "parallel")
    broken(lambda c: c["layers"][0]["mixer"].pop("mask"), "mask")
    broken(lambda c: c["layers"][0]["mixer"].pop("q_rank"), "q_rank")
    broken(lambda c: c["layers"][0]["mixer"]["rot"].update(dims=14), "rot_dim")
    broken(lambda c: c["layers"][0]["mixer"]["rot"].update(dims=11), "odd")
    broken(lambda c: c["layers"][1]["mixer"].update(heads=0), "heads")
    broken(lambda c: c["layers"][2]["mixer"].update(kv_heads=4), "kv_heads")
    broken(lambda c: c["layers"][2]["mlp"].update(kind="moe"), "kind")
    broken(lambda c: c["layers"][5]["mlp"].pop("ff"), "ff")
