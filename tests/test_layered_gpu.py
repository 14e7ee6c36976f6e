"""Layered designs on the GPU against their plain statement (oracle/layered.py), through the library's own entry points: Timerax's mechanisms
one by one (Ranutar's are in test_ranutar_gpu.py), then both whole designs.

32-bit runs are held to 1e-5 of the residual stream's (or the logits') scale, bfloat16 runs to a few percent.  The models are tiny,
have random weights and sizes that no other file uses; attention scales are large enough for single keys to dominate, so that a key
too many or too few shows."""
import copy
import json
import os
import subprocess

import numpy as np
import pytest

from oracle import layered as O
from tests import layered_util as U

pytestmark = pytest.mark.gpu
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
F32, B16 = U.F32, U.B16


@pytest.fixture(params=[U.mixed, U.sandwich_mixed], ids=["Timerax", "Ranutar"])
def design(request):
    """a configuration with every mechanism of a design"""
    return request.param


def only_left(W):   # the recurrent half of every pair silenced
    for k in W:
        if k.endswith("right.out"):
            W[k][:] = 0


def only_right(W):
    for k in W:
        if k.endswith("left.out"):
            W[k][:] = 0


def no_mixers(W):
    for k in W:
        if k.endswith("left.out") or k.endswith("right.out"):
            W[k][:] = 0


def check_trace(K, n, tol=None, cuts=()):
    K.check_trace(n, tol, cuts)


# ---- each mechanism alone ------------------------------------------------------------------------------------
@pytest.mark.parametrize("a", [
    U.attn(4, 2, 40, 24, 19, 0.4, 16), U.attn(3, 3, 32, 32, 64, 1.0, 32, yarn=False), U.attn(8, 1, 18, 10, 7, 2.0, 18),
    U.attn(2, 2, 130, 100, 33, 0.2, 64, 5e5), U.attn(2, 1, 256, 256, 50, 0.1, 2), U.attn(5, 5, 64, 33, 1, 1.0, 64)],
    ids=["grouped", "no-yarn", "one-kv-head", "wide-heads", "256", "chunk-1"])
def test_chunked_attention_alone(case, a):
    K = case(U.config([U.parallel(left=a)]), edit=only_left)
    check_trace(K, 150, cuts=([75], [1, 3, 5], [a["mask"]["size"]], list(range(130, 150))))


@pytest.mark.parametrize("m", [U.mlstm(3, 20, 28, 9.0), U.mlstm(1, 64, 64, 15.0), U.mlstm(2, 130, 70, 3.0), U.mlstm(2, 256, 256, 12.0), U.mlstm(5, 3, 1, 6.0)],
                         ids=["odd", "64", "two-groups", "256", "tiny"])
@pytest.mark.parametrize("bias", [0.0, 8.0, -8.0])
def test_mlstm_alone(case, m, bias):
    def edit(W):
        only_right(W)
        W["l0.mix.right.i.b"][:] += bias
    K = case(U.config([U.parallel(right=m)], width=72, eps=0.05), edit=edit)  # (the norm behind it hides the normaliser at a small eps)
    check_trace(K, 90, tol=3e-5, cuts=([37], [2, 4], list(range(70, 90))))


@pytest.mark.parametrize("d", [U.delta(6, 2, 24, 40, 4), U.delta(2, 2, 128, 128, 3), U.delta(3, 3, 60, 130, 2), U.delta(2, 1, 256, 256, 4),
                               U.delta(4, 2, 7, 5, 1), U.delta(2, 2, 33, 64, 6)],
                         ids=["grouped", "128", "two-groups", "256", "no-conv", "6-taps"])
def test_delta_rule_alone(case, d):
    K = case(U.config([U.channel_delta(d)], width=88))
    check_trace(K, 90, cuts=([41], [1, 2, 3], list(range(70, 90))))


@pytest.mark.parametrize("rate", [-6.0, 3.5])
def test_delta_rule_with_slow_and_with_violent_decays(case, rate):
    def edit(W):
        W["l0.mix.A_log"][:] = rate
        W["l0.mix.dt_bias"][::2] += 4.0
    K = case(U.config([U.channel_delta()]), edit=edit)
    check_trace(K, 60, cuts=([20],))


def test_delta_rule_with_repeated_keys(case):
    """the same key again and again, no decay, full steps: the triangular system of a chunk at its worst"""
    def edit(W):
        W["l0.mix.A_log"][:] = -12.0
        W["l0.mix.b"][:] *= 0.0
        W["embed"][:] = U.bf16(W["embed"][:1] + 0.02 * W["embed"])
    K = case(U.config([U.channel_delta()]), edit=edit)
    check_trace(K, 80, tol=5e-5, cuts=([33],))


@pytest.mark.parametrize("m", [U.moe(7, 3, 40, 0.8, 72, 1.2), U.moe(5, 1, 24, 1.0, 0), U.moe(4, 4, 130, 0.3, 16, 2.0), U.moe(150, 9, 8, 1.0, 8)],
                         ids=["shared", "top-1", "all", "many"])
def test_experts_alone(case, m):
    K = case(U.config([U.parallel(mlp=m)]), edit=no_mixers)
    check_trace(K, 200, cuts=([50], list(range(180, 200))))


def test_logits_without_and_with_a_soft_cap(case):
    c = U.config([U.channel_delta()], softcap=3.0)
    K = case(c)
    assert np.abs(K.got(K.tokens(9))).max() <= 3.0
    check_trace(K, 9)
    c = copy.deepcopy(c)
    del c["logit_softcap"]
    c["logit_softcap"] = 1e9  # (the oracle always caps: a cap far away is none)
    check_trace(case(c), 9)


# ---- the whole design ------------------------------------------------------------------------------------------
@pytest.mark.parametrize("width", [120, 64, 77, 300], ids=lambda w: f"width-{w}")
def test_all_layers_in_32_bit(design, case, width):
    check_trace(case(design(width), seed=width), 100, tol=2e-5, cuts=([64], [2, 4, 6, 8], [19, 38, 57]))


def test_bfloat16_stays_close(design, case):
    K = case(design(), dtype="bfloat16")
    t = K.tokens(100)
    want = K.want(t)
    for got in (K.got(t), K.got(t, range(40, 100))):
        assert U.err(got, want, 0.8) < K.tol and U.err(got, want) < 0.5  # (a close call of a router may go the other way)


@pytest.mark.parametrize("size", [2, 3, 7, 16, 17, 33, 64])
def test_portions_of_a_prompt(design, case, size):
    K = case(design())
    t = K.tokens(130)
    assert U.err(K.got(t, range(size, 130, size)), K.want(t)) < 2e-5


def test_portions_larger_than_one_pass(design, case):
    K = case(design(), options="piece_tokens=48")
    t = K.tokens(131)
    assert U.err(K.got(t), K.want(t)) < 2e-5
    assert U.err(K.got(t, [100]), K.want(t)) < 2e-5


@pytest.mark.parametrize("options", ["fused_decode=0", "decode_graph=0", "chunk_scan=0", "fused_decode=0,decode_graph=0,chunk_scan=0"])
def test_every_option_computes_the_same(design, case, options):
    K, L = case(design()), case(design(), options=options)
    t = K.tokens(70)
    a, b = K.got(t, range(40, 70)), L.got(t, range(40, 70))
    assert U.err(a, b) < 2e-5
    assert (L.lm.info("fused_decode_layers") == 0) == ("fused_decode=0" in options)
    assert (L.lm.info("graph_captured") == 0) == ("decode_graph=0" in options)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_unequal_requests_together_and_alone(design, case, dtype):
    K = case(design(), dtype=dtype)
    lens = [1, 37, 64, 5, 20]
    toks = [K.tokens(n + 25, seed=n) for n in lens]
    seqs = [K.lm.seq_open() for _ in lens]
    logits = K.lm.step([(s, t[:n], range(n)) for s, t, n in zip(seqs, toks, lens)])
    got = [list(p) for p in np.split(logits, np.cumsum(lens)[:-1])]
    live = list(range(5))
    for i in range(25):
        step = K.lm.step([(seqs[j], [toks[j][lens[j] + i]], [0]) for j in live])
        for j, row in zip(live, step):
            got[j].append(row)
        if i % 6 == 5 and len(live) > 1:   # shorter requests end earlier
            K.lm.seq_close(seqs[live.pop(0)])
    for j in range(5):
        n = len(got[j])
        alone = K.got(toks[j][:n], range(lens[j], n))
        part, tol = (1.0, 2e-5) if dtype == "float32" else (0.8, B16)
        assert U.err(np.array(got[j]), K.want(toks[j][:n]), part) < tol
        assert U.err(np.array(got[j]), alone, part) < tol


def test_more_sequences_than_one_decode_launch_takes(design, case):
    K = case(design())
    toks = [K.tokens(12, seed=n) for n in range(21)]
    seqs = [K.lm.seq_open() for _ in toks]
    K.lm.step([(s, t[:8], []) for s, t in zip(seqs, toks)])
    for i in range(8, 12):
        got = K.lm.step([(s, [t[i]], [0]) for s, t in zip(seqs, toks)])
    for t, row in zip(toks, got):
        assert U.err(row[None], K.want(t)[-1:]) < 2e-5


def test_slots_are_used_again_without_a_trace_of_what_they_held(design, case):
    K = case(design())
    t = K.tokens(50, seed=5)
    fresh = K.got(t, range(30, 50))
    seqs = [K.lm.seq_open() for _ in range(6)]
    for i, s in enumerate(seqs):
        K.lm.step([(s, K.tokens(40 + i, seed=40 + i), [])])
        K.lm.step([(s, [3], [])])
    slots = K.lm.info("sequence_slots")
    for s in seqs:
        K.lm.seq_close(s)
    assert K.lm.info("live_sequences") == 0
    for _ in range(3):
        assert np.array_equal(K.got(t, range(30, 50)), fresh)
    assert K.lm.info("sequence_slots") == slots
    with pytest.raises(Exception, match="not open"):
        K.lm.step([(seqs[0], [1], [])])


# ---- chunk edges ---------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("chunk", [16, 31, 32, 33, 64, 128, 130, 300])
def test_chunk_edges_in_prompts_and_in_decoding(case, chunk):
    """scores so steep that one key decides: the first key of a chunk is seen by its whole chunk and by nobody behind it"""
    def edit(W):
        only_left(W)
        W["embed"][7] = U.bf16(6 * W["embed"][7])
    K = case(U.config([U.parallel(left=U.attn(4, 2, 32, 32, chunk, 1.5, 16))]), edit=edit)
    n = 2 * chunk + 5
    t = K.tokens(n)
    for p in (0, chunk - 1, chunk, 2 * chunk - 1, 2 * chunk):
        t[p] = 7
    want = K.want(t)
    for cuts in ([], [chunk - 1], [chunk], [chunk + 1], list(range(chunk - 3, chunk + 4)), list(range(2 * chunk - 2, n))):
        got = K.got(t, cuts)
        assert U.err(got, want) < 2e-5, cuts


def test_attention_parts_meet_in_decoding(case):
    """a chunk of several hundred keys: decode steps deal it to several workgroups, with another graph per power of two"""
    K = case(U.config([U.parallel(left=U.attn(4, 1, 48, 40, 700, 0.5, 48), mlp=U.moe())]))
    t = K.tokens(620)
    want = K.want(t)
    for start in (120, 250, 600):
        assert U.err(K.got(t[:start + 20], [start] + list(range(start + 1, start + 20))), want[:start + 20]) < 2e-5
    assert K.lm.info("graph_captured") >= 3


def test_long_decoding(design, case):
    K = case(design())
    t = K.tokens(260)
    assert U.err(K.got(t, range(3, 260)), K.want(t)) < 3e-5
    assert K.lm.info("graph_steps") > 200


def test_first_tokens(design, case):
    K = case(design())
    t = K.tokens(6)
    want = K.want(t)
    for cuts in ([], [1], [1, 2], [1, 2, 3, 4, 5], [2, 3]):
        assert U.err(K.got(t, cuts), want) < 2e-5


# ---- entry points ----------------------------------------------------------------------------------------------------
def test_single_sequence_calls(design, case):
    import dsk
    K = case(design())
    t = K.tokens(30)
    want = K.want(t)
    assert U.err(K.lm.hydrate(t[:20], 0, dsk.MODE_OUTPUT_LOGITS)[None], want[19:20]) < 2e-5
    for i in range(20, 28):
        assert U.err(K.lm.forward(int(t[i]), i)[None], want[i:i + 1]) < 2e-5
    assert K.lm.forward_argmax(int(t[28]), 28) == want[28].argmax()
    p = np.exp(want[29] - want[29].max())
    assert K.lm.forward_prob(int(t[29]), 29, 5) == pytest.approx(p[5] / p.sum(), rel=1e-3)
    with pytest.raises(dsk.DskError, match="stands at"):
        K.lm.forward(1, 4)
    assert U.err(K.lm.forward(int(t[0]), 0)[None], want[:1]) < 2e-5   # position 0 starts anew


def test_sampling_follows_the_sampler(design, case, ctx):
    K = case(design())
    t = K.tokens(15)
    coins = np.linspace(0.02, 0.98, 7).astype(np.float32)
    for temperature, top_p in ((0.0, 1.0), (1.0, 1.0), (2.5, 0.9)):
        seqs = [K.lm.seq_open() for _ in range(7)]
        K.lm.step([(s, t[i:i + 8], []) for i, s in enumerate(seqs)])
        twins = [K.lm.seq_open() for _ in range(7)]
        K.lm.step([(s, t[i:i + 8], []) for i, s in enumerate(twins)])
        for _ in range(3):   # eager, captured, replayed
            nxt = K.lm.step_sample([(s, [11]) for s in seqs], temperature, top_p, coins)
            lg = K.lm.step([(s, [11], [0]) for s in twins])
            assert list(nxt) == [ctx.sample(lg[i], temperature, top_p, float(coins[i])) for i in range(7)]
        for s in seqs + twins:
            K.lm.seq_close(s)


def test_greedy_generation(design, case):
    K = case(design())
    prompts = [K.tokens(n, seed=n) for n in (1, 9, 30, 4, 17)]
    news = [12, 20, 7, 1, 16]
    for max_batch in (16, 2):
        got = K.lm.generate(prompts, news, max_batch=max_batch)
        for p, n, g in zip(prompts, news, got):
            assert len(g) == n
            s = O.Sequence(K.ref)
            lg = K.ref.run(s, p)[-1]
            for tok in g:
                assert lg[tok] > lg.max() - 1e-4 * np.abs(lg).max()   # (a tie to rounding may go either way)
                lg = K.ref.run(s, [tok])[-1]
    assert K.lm.info("live_sequences") == 0
    stop = got[1][3]
    cut = K.lm.generate(prompts, news, stop_token=stop)
    assert cut[1] == got[1][:got[1].index(stop) + 1]
    assert K.lm.generate(prompts[:2], 5, temperature=0.8, seed=3) == K.lm.generate(prompts[:2], 5, temperature=0.8, seed=3)


def test_bad_weights_and_steps_are_errors(case, ctx, tmp_path):
    import dsk
    K = case(U.mixed())
    W = dict(K.W)
    W["l1.mix.q"] = W["l1.mix.q"][:-1]
    with pytest.raises(dsk.DskError, match="l1.mix.q"):
        dsk.LM(ctx, U.save(tmp_path / "short", K.c, W))
    del W["l1.mix.q"]
    with pytest.raises(dsk.DskError, match="l1.mix.q is missing"):
        dsk.LM(ctx, U.save(tmp_path / "gone", K.c, W))
    with pytest.raises(dsk.DskError, match="option"):
        dsk.LM(ctx, K.dir, options="no_such=1")
    s = K.lm.seq_open()
    with pytest.raises(dsk.DskError, match="out of range"):
        K.lm.step([(s, [K.c["vocab"]], [])])
    with pytest.raises(dsk.DskError, match="twice"):
        K.lm.step([(s, [1], []), (s, [2], [])])
    with pytest.raises(dsk.DskError, match="DeepSeek"):
        dsk.check(dsk.lib().dsk_model_finalize(K.lm.h))
    assert K.lm.seq_pos(s) == 0


def test_trace_runner(design, case, tmp_path):
    K = case(design())
    a, b = K.tokens(12, 1), K.tokens(9, 2)
    steps = [{"step": 0, "entries": [{"id": "x", "tokens": a[:10].tolist(), "want": [9, 0]}, {"id": "y", "tokens": b[:7].tolist(), "want": []}], "end": []},
             {"step": 1, "entries": [{"id": "x", "tokens": a[10:11].tolist(), "want": []}, {"id": "y", "tokens": b[7:8].tolist(), "want": []}], "end": []},
             {"step": 2, "entries": [{"id": "x", "tokens": a[11:12].tolist(), "want": [0]}, {"id": "y", "tokens": b[8:9].tolist(), "want": [0]}], "end": ["x", "y"]},
             {"step": 3, "entries": [{"id": "x", "tokens": b[:3].tolist(), "want": [2]}], "end": ["x"]}]
    out = tmp_path / "out"
    out.mkdir()
    r = subprocess.run([os.path.join(ROOT, "bin", "trace_run"), "--model", K.dir, "--dtype", "float32", "--out", str(out), "--max-tokens", "64"],
                       input="".join(json.dumps(s) + "\n" for s in steps).encode(), capture_output=True, timeout=110)
    assert r.returncode == 0, r.stderr.decode()[-2000:]
    assert [l for l in r.stdout.decode().splitlines() if l.startswith("done")] == [f"done {i}" for i in range(4)]
    V = K.c["vocab"]
    wa, wb = K.want(a), K.want(b)

    def read(n):
        return np.fromfile(out / f"{n}.f32", "<f4").reshape(-1, V)
    assert U.err(read(0), wa[[9, 0]]) < 2e-5 and not (out / "1.f32").exists()
    assert U.err(read(2), np.array([wa[11], wb[8]])) < 2e-5 and U.err(read(3), wb[2:3]) < 2e-5


def test_generate_command(design, case):
    K = case(design())
    prompts = [K.tokens(5, 1).tolist(), K.tokens(11, 2).tolist()]
    r = subprocess.run([os.path.join(ROOT, "bin", "generate"), "--model", K.dir, "--dtype", "float32", "-n", "6"] + [",".join(map(str, p)) for p in prompts],
                       capture_output=True, timeout=110)
    assert r.returncode == 0, r.stderr.decode()[-2000:]
    got = [[int(v) for v in l.split(",")] for l in r.stdout.decode().split()]
    assert got == K.lm.generate(prompts, 6)


def test_deepseek_checkpoints_answer_the_same_calls(ctx):
    """the other family behind the same handle: steps, sequences and greedy generation of a .dseek directory"""
    import dsk
    d = os.path.join(ROOT, "tests", "golden", "converted_f8e5m2")
    A, B = dsk.Model.from_dseek(ctx, d), dsk.LM(ctx, d)
    assert B.family == "deepseek" and B.vocab == A.cfg.vocab_size
    t = np.random.default_rng(0).integers(0, B.vocab, 9)
    want = [A.forward(int(x), i) for i, x in enumerate(t)]
    s = B.seq_open()
    got = B.step([(s, t, [2, 8])])
    assert np.array_equal(got, np.array([want[2], want[8]]))
    with pytest.raises(dsk.DskError, match="one sequence"):
        B.seq_open()
    B.seq_close(s)
    out = B.generate([t[:5], t[3:6]], 4, max_batch=1)
    x, pos = int(t[4]), 4
    for i, y in enumerate(t[:4]):
        A.forward(int(y), i, dsk.MODE_HYDRATE_KV_CACHE)
    for y in out[0]:
        assert A.forward_argmax(x, pos) == y
        x, pos = y, pos + 1
    A.close()
    B.close()
