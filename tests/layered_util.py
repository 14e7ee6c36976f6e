"""Small configurations, random weights and files of layered designs for the tests (the plain statement of the design is
oracle/layered.py)."""
import copy
import json
import os
import struct

import numpy as np

from oracle import layered as O

F32, B16 = 1e-5, 0.06  # tolerances: of the residual stream's (or the logits') scale


class Case:
    """one model on both sides: the library's (lm) and the plain statement's (ref)"""

    def __init__(self, ctx, tmp, c, seed=0, dtype="float32", options=None, edit=None, **kw):
        import dsk
        self.c, self.W = c, weights(c, seed, **kw)
        if edit:
            edit(self.W)
            self.W = {k: bf16(v) for k, v in self.W.items()}
        self.dir = save(tmp, c, self.W)
        self.lm = dsk.LM(ctx, self.dir, dtype, options)
        self.ref = O.Model(c, self.W)
        self.tol = F32 if dtype == "float32" else B16

    def tokens(self, n, seed=1):
        return np.random.default_rng(seed).integers(0, self.c["vocab"], n)

    def want(self, tokens):
        return self.ref.run(O.Sequence(self.ref), tokens)

    def got(self, tokens, cuts=()):
        """logits of one sequence run in portions"""
        s = self.lm.seq_open()
        out = [self.lm.step([(s, p, range(len(p)))]) for p in np.split(np.asarray(tokens), list(cuts)) if len(p)]
        assert self.lm.seq_pos(s) == len(tokens)
        self.lm.seq_close(s)
        return np.concatenate(out)

    def check_trace(self, n, tol=None, cuts=()):
        """residual stream behind every layer, prompt in one step; then logits, also cut"""
        t, trace, tol = self.tokens(n), [], tol or self.tol
        want = self.ref.run(O.Sequence(self.ref), t, trace)
        self.lm.set_trace(True)
        s = self.lm.seq_open()
        got = self.lm.step([(s, t, range(n))])
        for l in range(len(self.c["layers"])):
            assert err(self.lm.trace_rows(l, n), trace[l]) < tol, l
        self.lm.seq_close(s)
        self.lm.set_trace(False)
        assert err(got, want) < tol
        for cut in cuts:
            assert err(self.got(t, cut), want) < tol, cut


def bf16(x):
    """round to bfloat16, as float32"""
    u = np.ascontiguousarray(x, np.float32).view(np.uint32)
    return ((u + 0x7FFF + ((u >> 16) & 1)) & 0xFFFF0000).view(np.float32)


def attn(heads=4, kv_heads=2, dim=40, vdim=24, chunk=19, scale=0.4, rot_dims=16, base=1000.0, yarn=True):
    rot = {"base": base, "dims": rot_dims}
    if yarn:
        rot["scaling"] = {"factor": 3.0, "original": 64, "fast": 8.0, "slow": 0.5}
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "mask": {"size": chunk}, "scale": scale, "rot": rot}


def mlstm(heads=3, dim=20, vdim=28, cap=9.0):
    return {"heads": heads, "dim": dim, "vdim": vdim, "gate_cap": cap}


def delta(heads=6, kv_heads=2, dim=24, vdim=40, conv=4):
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv}


def moe(experts=7, top=3, ff=40, limit=0.8, shared=72, shared_limit=1.2):
    m = {"kind": "moe", "router": {"experts": experts, "top": top}, "expert": {"ff": ff, "limit": limit}}
    if shared:
        m["shared"] = {"ff": shared, "limit": shared_limit}
    return m


def parallel(left=None, right=None, mlp=None):
    return {"type": "parallel", "mixer": {"left": left or attn(), "right": right or mlstm()}, "mlp": mlp}


def channel_delta(mixer=None, mlp=None):
    return {"type": "channel_delta", "mixer": mixer or delta(), "mlp": mlp}


def config(layers, width=120, vocab=203, eps=1e-5, softcap=20.0):
    return {"architecture": "Timerax", "width": width, "vocab": vocab, "norm": {"eps": eps}, "logit_softcap": softcap, "layers": copy.deepcopy(layers)}


def mixed(width=120, **kw):
    """every mechanism, sizes that are all different"""
    return config([parallel(mlp=moe()), channel_delta(mlp=moe(experts=9, top=2, ff=56, shared=0)), parallel(attn(6, 3, 32, 48, 32), mlstm(5, 36, 16), None),
                   channel_delta(delta(4, 4, 48, 32, 3), moe(5, 5, 24, 1.5, 40))], width=width, **kw)


def wkv(heads=3, dim=20):
    return {"type": "wkv", "mixer": {"heads": heads, "dim": dim}, "mlp": dense()}


def head_delta(*a, **kw):
    return {"type": "delta", "mixer": delta(*a, **kw), "mlp": dense()}


def latent(heads=5, dim=24, rot_dim=12, vdim=20, q_rank=36, kv_rank=28, window=13, scale=0.5, base=700.0, rot_dims=None):
    return {"type": "latent_attention", "mlp": dense(),
            "mixer": {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "q_rank": q_rank, "kv_rank": kv_rank, "mask": {"size": window},
                      "scale": scale, "rot": {"base": base, "dims": rot_dims or rot_dim}}}


def dense(ff=72):
    return {"kind": "dense", "ff": ff}


def no_ff(layer):
    return dict(layer, mlp=None)


def sandwich(layers, width=104, vocab=211, eps=1e-5, taps=4, logit_scale=0.7):
    return {"architecture": "Ranutar", "width": width, "vocab": vocab, "norm": {"eps": eps}, "canon": {"taps": taps}, "logit_scale": logit_scale,
            "layers": copy.deepcopy(layers)}


def sandwich_mixed(width=104, **kw):
    """every mechanism, sizes that are all different, windows shorter than the tests' prompts"""
    return sandwich([latent(), no_ff(wkv()), head_delta(6, 2, 24, 40, 4), dict(latent(2, 40, 34, 66, 50, 70, 37, 0.3), mlp=dense(130)), no_ff(head_delta(3, 3, 36, 20, 3)),
                     wkv(2, 52)], width=width, **kw)


def sandwich_weights(c, seed, rank):
    rng = np.random.default_rng(seed)
    D, W = c["width"], {}

    def mat(name, rows, cols, gain=1.0):
        W[name] = bf16(rng.normal(size=(rows, cols)) * gain / np.sqrt(cols))

    def vec(name, n, mean=0.0, std=0.3):
        W[name] = bf16(mean + std * rng.normal(size=n))
    W["embed"] = bf16(rng.normal(size=(c["vocab"], D)))
    vec("final.norm", D)
    mat("head", c["vocab"], D, 4.0)
    for i, L in enumerate(c["layers"]):
        p, m = f"l{i}.", L["mixer"]
        q = p + "mix"
        for n in ("1", "2")[:2 if L["mlp"] else 1]:
            vec(p + "norm" + n, D)
            vec(p + "norm" + n + "b", D)
            W[p + "canon" + n] = bf16(0.5 * rng.normal(size=(D, c["canon"]["taps"])))
        if L["type"] == "wkv":
            n = m["heads"] * m["dim"]
            for t in "rkvgw":
                W[f"{q}.mu.{t}"] = bf16(rng.uniform(0, 1, D))
            for t in "rkvg":
                mat(f"{q}.{t}", n, D)
            mat(q + ".w1", rank, D)
            mat(q + ".w2", n, rank)
            vec(q + ".w0", n, -1.5, 1.5)
            W[q + ".u"] = bf16(rng.normal(size=(m["heads"], m["dim"])))
            vec(q + ".norm", n, 1.0)
            mat(q + ".o", D, n)
        elif L["type"] == "delta":
            nq, nv = m["kv_heads"] * m["dim"], m["heads"] * m["vdim"]
            for t, n in (("q", nq), ("k", nq), ("v", nv)):
                mat(f"{q}.{t}", n, D)
                W[f"{q}.{t}.conv"] = bf16(rng.normal(size=(n, m["conv"])))
            mat(q + ".a", m["heads"], D)
            mat(q + ".b", m["heads"], D)
            W[q + ".A_log"] = bf16(np.log(rng.uniform(0.02, 1.5, m["heads"])))
            vec(q + ".dt_bias", m["heads"], -2.0, 1.5)
            vec(q + ".norm", m["vdim"], 1.0)
            mat(q + ".g", nv, D)
            mat(q + ".o", D, nv)
        else:
            mat(q + ".dq", m["q_rank"], D)
            vec(q + ".dq.norm", m["q_rank"], 1.0)
            mat(q + ".uq", m["heads"] * (m["dim"] + m["rot_dim"]), m["q_rank"])
            mat(q + ".dkv", m["kv_rank"] + m["rot_dim"], D)
            vec(q + ".dkv.norm", m["kv_rank"], 1.0)
            mat(q + ".uk", m["heads"] * m["dim"], m["kv_rank"])
            mat(q + ".uv", m["heads"] * m["vdim"], m["kv_rank"])
            mat(q + ".o", D, m["heads"] * m["vdim"])
        if L["mlp"]:
            mat(p + "mlp.up", L["mlp"]["ff"], D)
            mat(p + "mlp.down", D, L["mlp"]["ff"])
            vec(p + "mlp.act", 2, 0.4, 0.8)
    return W


def attract(W, token=7, seed=0, gain=6.0):
    """latent attention in layer 0: every query points (nearly) the same way, and the key of `token` along it, in all heads and by `gain` in the
    score; nobody else's does.  Whether `token` is seen decides the output."""
    rng = np.random.default_rng(seed)
    W["embed"][:, 0], W["embed"][:, 1], W["embed"][token, 1] = 3.0, 0.0, 8.0
    W["l0.norm1"][:] = 0.0
    for n in ("dq", "dkv"):
        W[f"l0.mix.{n}.norm"][:] = 1.0
    a = rng.normal(size=W["l0.mix.dq"].shape[0])
    W["l0.mix.dq"] *= 0.15
    W["l0.mix.dq"][:, 0] += a
    rank = W["l0.mix.uk"].shape[1]
    heads = W["attract.heads"]
    q = (W["l0.mix.uq"] @ (a / np.sqrt((a * a).mean()))).reshape(heads, -1)[:, :W["l0.mix.uk"].shape[0] // heads]
    k = W["l0.mix.uk"].reshape(heads, -1, rank)
    e = sum(k[h].T @ q[h] / np.linalg.norm(k[h].T @ q[h]) for h in range(heads))
    e /= np.sqrt((e * e).mean())
    W["l0.mix.dkv"][:rank, 1] = 2 * e
    return gain / min(q[h] @ k[h] @ e for h in range(heads))


def attracted(window, heads=4, seed=0):
    """(configuration, edit) of one latent attention layer in which token 7 stands out: its score is at least 6 in every head"""
    c = sandwich([no_ff(latent(heads, 32, 16, 24, 40, 48, window, 1.0))], taps=1)
    W = dict(weights(c, seed), **{"attract.heads": heads})
    c["layers"][0]["mixer"]["scale"] = float(attract(W))

    def edit(V):
        V["attract.heads"] = heads
        attract(V)
        del V["attract.heads"]
    return c, edit


def weights(c, seed=0, rank_a=12, rank_g=9):
    """random weights at which every mechanism has a say, rounded to bfloat16"""
    if c["architecture"] == "Ranutar":
        return sandwich_weights(c, seed, rank_a)
    rng = np.random.default_rng(seed)
    D, V, W = c["width"], c["vocab"], {}

    def mat(name, rows, cols, gain=1.0):
        W[name] = bf16(rng.normal(size=(rows, cols)) * gain / np.sqrt(cols))

    def vec(name, n, mean=0.0, std=0.3):
        W[name] = bf16(mean + std * rng.normal(size=n))
    W["embed"] = bf16(rng.normal(size=(V, D)))
    vec("final.norm", D)
    mat("head", V, D, 4.0)
    for i, L in enumerate(c["layers"]):
        p, m = f"l{i}.", L["mixer"]
        vec(p + "norm1", D)
        if L["type"] == "parallel":
            a, r = m["left"], m["right"]
            q = p + "mix.left"
            mat(q + ".q", a["heads"] * a["dim"], D)
            mat(q + ".k", a["kv_heads"] * a["dim"], D)
            mat(q + ".v", a["kv_heads"] * a["vdim"], D)
            mat(q + ".o", D, a["heads"] * a["vdim"])
            q = p + "mix.right"
            mat(q + ".q", r["heads"] * r["dim"], D)
            mat(q + ".k", r["heads"] * r["dim"], D)
            mat(q + ".v", r["heads"] * r["vdim"], D)
            mat(q + ".g", r["heads"] * r["vdim"], D)
            mat(q + ".o", D, r["heads"] * r["vdim"])
            vec(q + ".norm", r["heads"] * r["vdim"], 1.0)
            mat(q + ".i", r["heads"], D, 2.0)
            vec(q + ".i.b", r["heads"], -1.0, 1.0)
            mat(q + ".f", r["heads"], D, 1.0)
            vec(q + ".f.b", r["heads"], 3.0, 1.0)
            vec(p + "mix.left.out", D, 1.0)
            vec(p + "mix.right.out", D, 1.0)
        else:
            q = p + "mix"
            nq, nv = m["kv_heads"] * m["dim"], m["heads"] * m["vdim"]
            for t, n in (("q", nq), ("k", nq), ("v", nv)):
                mat(f"{q}.{t}", n, D)
                W[f"{q}.{t}.conv"] = bf16(rng.normal(size=(n, m["conv"])))
            mat(q + ".b", m["heads"], D)
            W[q + ".A_log"] = bf16(np.log(rng.uniform(0.02, 1.5, m["heads"])))
            vec(q + ".norm", m["vdim"], 1.0)
            mat(q + ".a1", rank_a, D)
            mat(q + ".a2", m["heads"] * m["dim"], rank_a)
            vec(q + ".dt_bias", m["heads"] * m["dim"], -2.0, 1.5)
            mat(q + ".g1", rank_g, D)
            mat(q + ".g2", nv, rank_g)
            mat(q + ".o", D, nv)
        e = L.get("mlp")
        if e:
            q = p + "mlp"
            for j in range(e["router"]["experts"]):
                mat(f"{q}.e{j}.gate", e["expert"]["ff"], D)
                mat(f"{q}.e{j}.up", e["expert"]["ff"], D)
                mat(f"{q}.e{j}.down", D, e["expert"]["ff"])
            mat(q + ".router", e["router"]["experts"], D, 3.0)
            if e.get("shared"):
                mat(q + ".shared.gate", e["shared"]["ff"], D)
                mat(q + ".shared.up", e["shared"]["ff"], D)
                mat(q + ".shared.down", D, e["shared"]["ff"])
    return W


def save(path, c, W):
    """config.json + model.safetensors (bfloat16)"""
    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(c, f)
    head, blobs, at = {}, [], 0
    for k, v in W.items():
        raw = (np.ascontiguousarray(v, np.float32).view(np.uint32) >> 16).astype("<u2").tobytes()
        head[k] = {"dtype": "BF16", "shape": list(v.shape), "data_offsets": [at, at + len(raw)]}
        blobs.append(raw)
        at += len(raw)
    js = json.dumps(head).encode()
    js += b" " * (-len(js) % 8)
    with open(os.path.join(path, "model.safetensors"), "wb") as f:
        f.write(struct.pack("<Q", len(js)) + js + b"".join(blobs))
    return str(path)


def err(got, want, part=1.0):
    """root mean square of the difference over that of the expectation: the worst row, or the worst of the best `part` of them"""
    got, want = np.asarray(got, np.float64), np.asarray(want, np.float64)
    return float(np.quantile(np.sqrt(((got - want) ** 2).mean(-1)) / np.sqrt((want ** 2).mean()), part))
