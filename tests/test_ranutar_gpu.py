"""The mechanisms of Ranutar on the GPU against their plain statement (oracle/layered.py): each one alone, with sizes, taps, windows and decays at
their ends, in prompts, portions, batches and decoding.  Whole models of the design run through test_layered_gpu.py.

32-bit runs, held to 1e-5 .. 3e-5 of the residual stream's (or the logits') scale.  Attention scores are steep, so that a key too many or
too few shows (test_ranutar_cpu.py plants such mistakes in the oracle)."""
import numpy as np
import pytest

from oracle import layered as O
from tests import layered_util as U

pytestmark = pytest.mark.gpu
TOL = 2e-5


def alone(layer, **kw):
    return U.sandwich([layer], **kw)


# ---- time mixing -------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("heads,dim,rank", [(3, 20, 12), (1, 16, 1), (2, 130, 40), (1, 256, 7), (5, 3, 70), (2, 64, 64)])
def test_time_mixing_alone(case, heads, dim, rank):
    K = case(alone(U.wkv(heads, dim), width=88), rank_a=rank)
    K.check_trace(90, cuts=([37], [1, 2, 4], list(range(70, 90)), list(range(2, 90, 2))))


@pytest.mark.parametrize("shift", [-9.0, 4.5])
def test_time_mixing_with_slow_and_with_violent_decays(case, shift):
    def edit(W):
        W["l0.mix.w0"][:] += shift
        W["l0.mix.w0"][::3] -= 2 * shift
    K = case(alone(U.no_ff(U.wkv(2, 36))), edit=edit)
    K.check_trace(75, tol=3e-5, cuts=([20], list(range(60, 75))))


def test_time_mixing_bonus_counts_for_the_current_token_only(case):
    def edit(W):
        W["l0.mix.u"][:] *= 20.0
    K = case(alone(U.no_ff(U.wkv(2, 36)), eps=0.05), edit=edit)
    K.check_trace(40, cuts=([1], [15, 16, 17], list(range(1, 40))))


def test_blends_with_the_previous_token(case):
    """nothing but the previous token in every blend: the first token blends with zero, a portion's first with the state"""
    def edit(W):
        for t in "rkvgw":
            W[f"l0.mix.mu.{t}"][:] = 1.0
    K = case(alone(U.no_ff(U.wkv()), eps=0.05), edit=edit)
    K.check_trace(50, cuts=([1], [16], [17, 18], list(range(30, 50))))


# ---- delta rule with a decay per head ------------------------------------------------------------------------------------
@pytest.mark.parametrize("d", [(6, 2, 24, 40, 4), (2, 2, 128, 128, 3), (3, 3, 60, 130, 2), (2, 1, 256, 256, 4), (4, 2, 7, 5, 1), (2, 2, 33, 64, 6), (1, 1, 16, 16, 5)], ids=str)
def test_delta_rule_alone(case, d):
    K = case(alone(U.head_delta(*d), width=88))
    K.check_trace(90, cuts=([41], [1, 2, 3], list(range(70, 90))))


@pytest.mark.parametrize("rate", [-6.0, 3.5])
def test_delta_rule_with_slow_and_with_violent_decays(case, rate):
    def edit(W):
        W["l0.mix.A_log"][:] = rate
        W["l0.mix.dt_bias"][::2] += 4.0
    case(alone(U.head_delta()), edit=edit).check_trace(60, cuts=([20], list(range(50, 60))))


def test_delta_rule_with_repeated_keys(case):
    """nearly the same key again and again, no decay, full steps: the triangular system of a chunk at its worst"""
    def edit(W):
        W["l0.mix.A_log"][:] = -12.0
        W["l0.mix.b"][:] *= 0.0
        W["embed"][:] = W["embed"][:1] + 0.02 * W["embed"]
    case(alone(U.head_delta(), taps=1), edit=edit).check_trace(80, tol=5e-5, cuts=([33],))


# ---- latent attention ------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("a", [
    U.latent(), U.latent(1, 16, 2, 16, 1, 1, 9), U.latent(3, 64, 32, 33, 64, 64, 50, 0.3), U.latent(2, 130, 64, 100, 200, 150, 33, 0.1), U.latent(17, 8, 8, 8, 24, 40, 21),
    U.latent(2, 192, 64, 256, 90, 512, 40, 0.1), U.latent(2, 5, 6, 3, 7, 9, 30, 1.0), U.latent(4, 32, 16, 24, 20, 20, 25, 0.5, rot_dims=10)],
    ids=["odd", "one-head", "64", "wide-heads", "17-heads", "largest", "tiny", "partly-rotated"])
def test_latent_attention_alone(case, a):
    K = case(alone(a))
    w = a["mixer"]["mask"]["size"]
    K.check_trace(150, cuts=([75], [1, 3, 5], [w, 2 * w], list(range(130, 150)), list(range(2, 150, 2))))


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("window", [1, 2, 3, 16, 31, 32, 33, 63, 64, 65, 96, 130, 200])
def test_window_edges_in_prompts_and_in_decoding(case, window, dtype):
    """one token outweighs all others as long as it is seen: just inside and just outside the window, at the edges of the kernels' tiles, in
    portions and decode steps on either side of the edge"""
    c, edit = U.attracted(window)
    K = case(c, edit=edit, dtype=dtype)
    for at in (0, 1, 31, 32, 64):
        n = at + window + 6
        t = K.tokens(n, seed=at)
        t[t == 7] = 8
        t[at] = 7
        want = K.want(t)
        last = at + window   # the first position that does not see it
        for cuts in ([], [last - 1], [last], [last + 1], [at, at + 1], list(range(max(1, last - 4), n)), [at + 1] + list(range(at + 3, n, 2))):
            assert U.err(K.got(t, sorted({c for c in cuts if c})), want) < (TOL if dtype == "float32" else U.B16), (at, cuts)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_parts_of_a_wide_window_meet_in_decoding(case, dtype):
    """a window of several hundred keys: decode steps deal it to several workgroups, with another graph per power of two"""
    K = case(alone(U.latent(6, 48, 32, 40, 70, 90, 600, 0.3)), dtype=dtype)
    t = K.tokens(640)
    want = K.want(t)
    for start in (20, 120, 250, 615):
        n = start + 20
        assert U.err(K.got(t[:n], [start] + list(range(start + 1, n))), want[:n]) < (TOL if dtype == "float32" else U.B16)
    assert K.lm.info("graph_captured") >= 4


def test_windows_of_several_sizes_and_small_passes(case):
    """portions that start with more old keys than one layer's ring holds, and steps that do not fit one pass"""
    K = case(U.sandwich([U.latent(window=5), U.latent(window=90), U.latent(window=33)]), options="piece_tokens=32")
    t = K.tokens(220)
    want = K.want(t)
    for cuts in ([], [100], [3, 95, 96, 98], list(range(40, 220, 40))):
        assert U.err(K.got(t, cuts), want) < TOL, cuts
    toks = [K.tokens(n, seed=n) for n in (130, 7, 100, 1, 60)]
    seqs = [K.lm.seq_open() for _ in toks]
    K.lm.step([(s, x[:len(x) // 2], []) for s, x in zip(seqs, toks) if len(x) > 1])
    got = K.lm.step([(s, x[len(x) // 2:], [len(x) - len(x) // 2 - 1]) for s, x in zip(seqs, toks)])
    assert U.err(got, np.array([K.want(x)[-1] for x in toks])) < TOL


def test_positions_far_from_the_start(case):
    K = case(alone(U.no_ff(U.latent(2, 16, 24, 16, 20, 24, 11, 0.3, base=900.0))))
    t = K.tokens(1500)
    want = K.want(t)
    assert U.err(K.got(t, [1000, 1001, 1450] + list(range(1451, 1500))), want) < 1e-4   # (angles in 32-bit: their rounding grows with the position)


# ---- around the mixers ---------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("taps", [1, 2, 3, 4, 5, 9])
@pytest.mark.parametrize("width", [72, 77])
def test_convolution_in_front_of_the_sublayers(case, taps, width):
    K = case(U.sandwich([U.wkv(), U.latent(window=400)], width=width, taps=taps))
    K.check_trace(60, cuts=([1], [1, 2, 3, 4, 5], [15, 16, 17, 33], list(range(40, 60)), list(range(2, 60, 2))))


@pytest.mark.parametrize("width", [64, 200, 1030, 2052])
def test_widths(case, width):
    case(U.sandwich([U.wkv(), U.head_delta()], width=width), seed=width).check_trace(40, cuts=([30, 31, 32],))


@pytest.mark.parametrize("p,q", [(3.0, -2.0), (-4.0, 2.5), (0.0, 0.0)])
def test_feed_forward(case, p, q):
    def edit(W):
        W["l0.mlp.act"][:] = [p, q]
        W["l0.mlp.up"][:] *= 3.0
    case(alone(dict(U.wkv(1, 8), mlp=U.dense(300))), edit=edit).check_trace(140, cuts=([139], list(range(130, 140))))


@pytest.mark.parametrize("ff", [576, 1152, 1184, 2112, 4100])
def test_products_split_over_k(case, ff):
    """down products (and a mixer's output product) long enough to be split into parts, of an odd and an even number of steps"""
    K = case(U.sandwich([dict(U.head_delta(9, 3, 8, 128, 4), mlp=U.dense(ff)), dict(U.wkv(2, 36), mlp=U.dense(ff))], width=88))
    K.check_trace(150, tol=TOL, cuts=([20], list(range(130, 150))))


@pytest.mark.parametrize("rows", [17, 300, 600])
def test_prompt_tiles_of_both_sizes(case, rows):
    c = U.sandwich([dict(U.wkv(4, 64), mlp=U.dense(1152)), dict(U.head_delta(5, 5, 64, 64, 4), mlp=U.dense(700)), U.latent(6, 64, 32, 48, 90, 130, 100, 0.1)], width=330)
    runs = [case(c, dtype="bfloat16", options=f"prompt_tile={tile}") for tile in (128, 256)]
    t = runs[0].tokens(rows)
    want = runs[0].want(t)
    a, b = (K.got(t) for K in runs)
    assert U.err(a, want) < U.B16 and U.err(b, want) < U.B16 and U.err(a, b) < U.B16


def test_layers_without_a_feed_forward_in_any_order(case):
    K = case(U.sandwich([U.no_ff(U.head_delta()), U.no_ff(U.latent()), U.wkv(), U.no_ff(U.wkv(1, 24)), U.latent(2, 16, 8, 16, 12, 20, 6)]))
    K.check_trace(60, tol=TOL, cuts=([9], list(range(50, 60))))


@pytest.mark.parametrize("scale", [1.0, 0.125, 3.0])
def test_scale_of_the_logits(case, scale):
    K = case(U.sandwich([U.no_ff(U.wkv())], logit_scale=scale))
    t = K.tokens(30)
    assert U.err(K.got(t), K.want(t)) < U.F32


# ---- passes of every kind -----------------------------------------------------------------------------------------------------------
def test_a_step_of_portions_and_single_tokens(case):
    """some sequences bring one token, some a portion, some begin; more single tokens than one decode launch takes"""
    K = case(U.sandwich_mixed())
    toks = [K.tokens(60, seed=n) for n in range(24)]
    seqs = [K.lm.seq_open() for _ in toks]
    done = [0 if i % 5 == 4 else 20 + i for i in range(24)]
    K.lm.step([(s, t[:d], []) for s, t, d in zip(seqs, toks, done) if d])
    for rnd in range(3):
        take = [(7 if i == rnd else 3 if i == 5 else 1) for i in range(24)]
        got = K.lm.step([(s, t[d:d + n], [n - 1]) for s, t, d, n in zip(seqs, toks, done, take)])
        done = [d + n for d, n in zip(done, take)]
        assert U.err(got, np.array([K.want(t[:d])[-1] for t, d in zip(toks, done)])) < TOL


@pytest.mark.parametrize("options", ["fused_decode=0", "chunk_scan=0"])
def test_every_path_of_every_mechanism(case, options):
    K = case(U.sandwich_mixed(), options=options)
    t = K.tokens(80)
    assert U.err(K.got(t, [50, 52] + list(range(53, 80))), K.want(t)) < TOL


def test_bad_weights_are_errors(case, ctx, tmp_path):
    import dsk
    K = case(U.sandwich_mixed())
    for name, cut in (("l0.mix.uk", 1), ("l1.mix.mu.g", 1), ("l0.canon2", 1), ("l2.mix.a", 1), ("l0.mlp.act", 1)):
        W = dict(K.W)
        W[name] = W[name][:-cut]
        with pytest.raises(dsk.DskError, match=name):
            dsk.LM(ctx, U.save(tmp_path / "short", K.c, W))
        del W[name]
        with pytest.raises(dsk.DskError, match=name + " is missing"):
            dsk.LM(ctx, U.save(tmp_path / "gone", K.c, W))
