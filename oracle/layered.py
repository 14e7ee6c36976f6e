"""Plain NumPy restatement of the layered (config-listed) model designs: the CPU side of their parity tests.

One function per mechanism, one token or one head at a time where that is the clearest statement, float64 throughout.
Nothing here is shared with the product: the product's kernels are checked AGAINST this file, so it reads the same
config.json keys and tensor names by itself and keeps no state besides what a mechanism's equations name.

Conventions: `W` maps tensor name -> array, linear weights are [out, in]; `p0` is the position of the first row of a
portion; every stateful mechanism takes its state dict and returns the outputs of the rows it was given, leaving the
state as the next portion needs it.
"""
import math

import numpy as np

F = np.float64


# ---- elementwise pieces ------------------------------------------------------------------------
def sigmoid(x):
    return np.where(x >= 0, 1 / (1 + np.exp(-np.abs(x))), np.exp(-np.abs(x)) / (1 + np.exp(-np.abs(x))))


def softplus(x):
    return np.maximum(x, 0) + np.log1p(np.exp(-np.abs(x)))


def logsigmoid(x):
    return -softplus(-x)


def silu(x):
    return x * sigmoid(x)


def rms(x, eps):
    """x over its root mean square along the last axis, eps inside the root"""
    return x / np.sqrt((x * x).mean(-1, keepdims=True) + eps)


def one_plus_norm(x, w, eps):
    """RMS norm whose weight is stored around zero"""
    return rms(x, eps) * (1 + w)


def xielu(z, p, q):
    """quadratic above zero, exponential below, the two halves with a common slope at zero; p and q through softplus"""
    return np.where(z > 0, softplus(p) * z * z, (0.5 + softplus(q)) * (np.expm1(np.minimum(z, 0)) - z)) + 0.5 * z


def unit(x):
    return x / np.sqrt((x * x).sum(-1, keepdims=True) + 1e-6)


# ---- rotary positions --------------------------------------------------------------------------
def yarn_frequencies(rot):
    """(frequencies [dims / 2], amplitude of cos and sin)"""
    dims, base = rot["dims"], float(rot["base"])
    i = np.arange(dims // 2, dtype=F)
    f = base ** (-2 * i / dims)
    sc = rot.get("scaling")
    if not sc:
        return f, 1.0

    def index_of(turns):
        return dims * math.log(sc["original"] / (2 * math.pi * turns)) / (2 * math.log(base))
    lo = max(math.floor(index_of(sc["fast"])), 0)
    hi = min(math.ceil(index_of(sc["slow"])), dims - 1)
    ramp = np.clip((i - lo) / max(hi - lo, 0.001), 0, 1)
    return f / sc["factor"] * ramp + f * (1 - ramp), 0.1 * math.log(sc["factor"]) + 1


def rotate_pairs(x, pos, rot):
    """interleaved pairs (2i, 2i + 1) of the first rot.dims dimensions; x [..., dim]"""
    f, amp = yarn_frequencies(rot)
    n = 2 * len(f)
    c, s = amp * np.cos(pos * f), amp * np.sin(pos * f)
    y = x.copy()
    u, v = x[..., 0:n:2], x[..., 1:n:2]
    y[..., 0:n:2] = u * c - v * s
    y[..., 1:n:2] = v * c + u * s
    return y


def rotate_halves(x, pos, rot):
    """pairs (i, i + dims / 2) of the first rot.dims dimensions; x [..., dim]"""
    n = rot["dims"] // 2
    a = pos * float(rot["base"]) ** (-2 * np.arange(n, dtype=F) / rot["dims"])
    y = x.copy()
    u, v = x[..., :n], x[..., n:2 * n]
    y[..., :n] = u * np.cos(a) - v * np.sin(a)
    y[..., n:2 * n] = v * np.cos(a) + u * np.sin(a)
    return y


# ---- chunked softmax attention -----------------------------------------------------------------
def chunked_attention(h, W, pre, m, eps, st, p0):
    H, G, dk, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    out = []
    for t, row in enumerate(h):
        pos = p0 + t
        q = (W[pre + ".q"] @ row).reshape(H, dk)
        k = (W[pre + ".k"] @ row).reshape(G, dk)
        v = (W[pre + ".v"] @ row).reshape(G, dv)
        q = rms(rotate_pairs(q, pos, m["rot"]), eps)
        k = rms(rotate_pairs(k, pos, m["rot"]), eps)
        st.setdefault("k", []).append(k)
        st.setdefault("v", []).append(v)
        first = pos // m["mask"]["size"] * m["mask"]["size"]
        o = np.zeros((H, dv))
        for n in range(H):
            g = n // (H // G)
            K = np.array([st["k"][j][g] for j in range(first, pos + 1)])
            V = np.array([st["v"][j][g] for j in range(first, pos + 1)])
            s = (K @ q[n]) * m["scale"]
            w = np.exp(s - s.max())
            o[n] = (w / w.sum()) @ V
        out.append(W[pre + ".o"] @ o.reshape(-1))
    return np.array(out)


# ---- mLSTM matrix memory -----------------------------------------------------------------------
def mlstm_step(S, n, m, q, k, v, i, f):
    """one head, one token: returns (S, n, m, o); S [dim, vdim]"""
    m1 = max(f + m, i)
    keep, add = math.exp(f + m - m1), math.exp(i - m1)
    S = keep * S + add * np.outer(k, v)
    n = keep * n + add * k
    o = (S.T @ q) / (max(abs(n @ q), math.exp(-m1)) + 1e-6)
    return S, n, m1, o


def mlstm(h, W, pre, m, eps, st):
    H, dk, dv, cap = m["heads"], m["dim"], m["vdim"], m["gate_cap"]
    if not st:
        st.update(S=np.zeros((H, dk, dv)), n=np.zeros((H, dk)), m=np.zeros(H))
    out = []
    for row in h:
        q = (W[pre + ".q"] @ row).reshape(H, dk) * dk ** -0.5
        k = (W[pre + ".k"] @ row).reshape(H, dk)
        v = (W[pre + ".v"] @ row).reshape(H, dv)
        i = cap * np.tanh((W[pre + ".i"] @ row + W[pre + ".i.b"]) / cap)
        f = logsigmoid(cap * np.tanh((W[pre + ".f"] @ row + W[pre + ".f.b"]) / cap))
        o = np.zeros((H, dv))
        for n in range(H):
            st["S"][n], st["n"][n], st["m"][n], o[n] = mlstm_step(st["S"][n], st["n"][n], st["m"][n], q[n], k[n], v[n], i[n], f[n])
        y = rms(o, eps).reshape(-1) * W[pre + ".norm"] * sigmoid(W[pre + ".g"] @ row)
        out.append(W[pre + ".o"] @ y)
    return np.array(out)


def parallel_mixer(h, W, pre, m, eps, st, p0):
    a = chunked_attention(h, W, pre + ".left", m["left"], eps, st.setdefault("left", {}), p0)
    b = mlstm(h, W, pre + ".right", m["right"], eps, st.setdefault("right", {}))
    return 0.5 * (rms(a, eps) * W[pre + ".left.out"] + rms(b, eps) * W[pre + ".right.out"])


# ---- gated delta rule with a decay per key channel ----------------------------------------------
def short_conv(x, taps_w, hist):
    """x [channels] of this token, hist [taps - 1, channels] (oldest first); returns (silu(conv), next hist)"""
    full = np.concatenate([hist, x[None]], 0)
    return silu((full * taps_w.T).sum(0)), full[1:]


def delta_step(S, q, k, v, g, beta):
    """one head, one token; S [dim, vdim], g [dim]"""
    S = g[:, None] * S
    u = beta * (v - S.T @ k)
    S = S + np.outer(k, u)
    return S, S.T @ q


def channel_delta(h, W, pre, m, eps, st):
    H, G, dk, dv, taps = m["heads"], m["kv_heads"], m["dim"], m["vdim"], m["conv"]
    if not st:
        st.update(S=np.zeros((H, dk, dv)), q=np.zeros((taps - 1, G * dk)), k=np.zeros((taps - 1, G * dk)), v=np.zeros((taps - 1, H * dv)))
    A = np.exp(W[pre + ".A_log"])
    out = []
    for row in h:
        q, st["q"] = short_conv(W[pre + ".q"] @ row, W[pre + ".q.conv"], st["q"])
        k, st["k"] = short_conv(W[pre + ".k"] @ row, W[pre + ".k.conv"], st["k"])
        v, st["v"] = short_conv(W[pre + ".v"] @ row, W[pre + ".v.conv"], st["v"])
        q, k, v = unit(q.reshape(G, dk)) * dk ** -0.5, unit(k.reshape(G, dk)), v.reshape(H, dv)
        beta = sigmoid(W[pre + ".b"] @ row)
        a = softplus(W[pre + ".a2"] @ (W[pre + ".a1"] @ row) + W[pre + ".dt_bias"]).reshape(H, dk)
        g = np.exp(-A[:, None] * a)
        o = np.zeros((H, dv))
        for n in range(H):
            kv = n // (H // G)
            st["S"][n], o[n] = delta_step(st["S"][n], q[kv], k[kv], v[n], g[n], beta[n])
        y = rms(o, eps) * W[pre + ".norm"]
        y = y.reshape(-1) * sigmoid(W[pre + ".g2"] @ (W[pre + ".g1"] @ row))
        out.append(W[pre + ".o"] @ y)
    return np.array(out)


# ---- gated delta rule with one decay per head -----------------------------------------------------
def head_delta(h, W, pre, m, eps, st):
    H, G, dk, dv, taps = m["heads"], m["kv_heads"], m["dim"], m["vdim"], m["conv"]
    if not st:
        st.update(S=np.zeros((H, dk, dv)), q=np.zeros((taps - 1, G * dk)), k=np.zeros((taps - 1, G * dk)), v=np.zeros((taps - 1, H * dv)))
    out = []
    for row in h:
        q, st["q"] = short_conv(W[pre + ".q"] @ row, W[pre + ".q.conv"], st["q"])
        k, st["k"] = short_conv(W[pre + ".k"] @ row, W[pre + ".k.conv"], st["k"])
        v, st["v"] = short_conv(W[pre + ".v"] @ row, W[pre + ".v.conv"], st["v"])
        q, k, v = unit(q.reshape(G, dk)) * dk ** -0.5, unit(k.reshape(G, dk)), v.reshape(H, dv)
        beta = sigmoid(W[pre + ".b"] @ row)
        g = np.exp(-np.exp(W[pre + ".A_log"]) * softplus(W[pre + ".a"] @ row + W[pre + ".dt_bias"]))
        o = np.zeros((H, dv))
        for n in range(H):
            kv = n // (H // G)
            st["S"][n], o[n] = delta_step(st["S"][n], q[kv], k[kv], v[n], np.full(dk, g[n]), beta[n])
        y = (rms(o, eps) * W[pre + ".norm"]).reshape(-1) * silu(W[pre + ".g"] @ row)
        out.append(W[pre + ".o"] @ y)
    return np.array(out)


# ---- time mixing with a decay per key channel and a bonus for the current token --------------------
def wkv_step(S, r, k, v, w, u):
    """one head, one token; S [dim, dim]"""
    o = (S + np.outer(u * k, v)).T @ r
    return w[:, None] * S + np.outer(k, v), o


def wkv(h, W, pre, m, eps, st):
    H, d = m["heads"], m["dim"]
    if not st:
        st.update(S=np.zeros((H, d, d)), h=np.zeros(h.shape[1]))
    out = []
    for row in h:
        mix = {s: row + (st["h"] - row) * W[f"{pre}.mu.{s}"] for s in "rkvgw"}
        st["h"] = row
        r, k, v = ((W[f"{pre}.{s}"] @ mix[s]).reshape(H, d) for s in "rkv")
        w = np.exp(-np.exp(W[pre + ".w2"] @ np.tanh(W[pre + ".w1"] @ mix["w"]) + W[pre + ".w0"])).reshape(H, d)
        o = np.zeros((H, d))
        for n in range(H):
            st["S"][n], o[n] = wkv_step(st["S"][n], r[n], k[n], v[n], w[n], W[pre + ".u"][n])
        out.append(W[pre + ".o"] @ (rms(o, eps).reshape(-1) * W[pre + ".norm"] * silu(W[pre + ".g"] @ mix["g"])))
    return np.array(out)


# ---- latent attention in a sliding window ----------------------------------------------------------
def latent_attention(h, W, pre, m, eps, st, p0):
    H, dk, dr, dv, rank = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    out = []
    for t, row in enumerate(h):
        pos = p0 + t
        q = (W[pre + ".uq"] @ (rms(W[pre + ".dq"] @ row, eps) * W[pre + ".dq.norm"])).reshape(H, dk + dr)
        kv = W[pre + ".dkv"] @ row
        st.setdefault("c", []).append(rms(kv[:rank], eps) * W[pre + ".dkv.norm"])
        st.setdefault("r", []).append(rotate_halves(kv[rank:], pos, m["rot"]))
        first = max(0, pos - m["mask"]["size"] + 1)
        C, R = np.array(st["c"][first:]), np.array(st["r"][first:])
        K = (C @ W[pre + ".uk"].T).reshape(-1, H, dk)
        V = (C @ W[pre + ".uv"].T).reshape(-1, H, dv)
        qr = rotate_halves(q[:, dk:], pos, m["rot"])
        o = np.zeros((H, dv))
        for n in range(H):
            s = (K[:, n] @ q[n, :dk] + R @ qr[n]) * m["scale"]
            w = np.exp(s - s.max())
            o[n] = (w / w.sum()) @ V[:, n]
        out.append(W[pre + ".o"] @ o.reshape(-1))
    return np.array(out)


# ---- causal convolution in front of a sublayer -----------------------------------------------------
def input_conv(h, w, st):
    """h + conv(h), the last taps - 1 rows of h kept; w [width, taps]"""
    taps = w.shape[1]
    full = np.concatenate([st.get("in", np.zeros((taps - 1, h.shape[1]))), h], 0)
    st["in"] = full[len(h):]
    return h + sum(full[j:j + len(h)] * w[:, j] for j in range(taps))


# ---- feed-forward ------------------------------------------------------------------------------
def clamped_glu(h, W, pre, limit):
    g = np.minimum(W[pre + ".gate"] @ h, limit)
    u = np.clip(W[pre + ".up"] @ h, -limit, limit)
    return W[pre + ".down"] @ (g * sigmoid(1.702 * g) * (u + 1))


def route(z, top):
    """(chosen experts, weights): the largest logits, the softmax over the chosen ones only"""
    e = np.argsort(-z, kind="stable")[:top]
    w = np.exp(z[e] - z[e].max())
    return e, w / w.sum()


def moe(h, W, pre, m):
    out = []
    for row in h:
        e, w = route(W[pre + ".router"] @ row, m["router"]["top"])
        y = sum(wi * clamped_glu(row, W, f"{pre}.e{ei}", m["expert"]["limit"]) for ei, wi in zip(e, w))
        if m.get("shared"):
            y = y + clamped_glu(row, W, pre + ".shared", m["shared"]["limit"])
        out.append(y)
    return np.array(out)


# ---- the models --------------------------------------------------------------------------------
class Sequence:
    """One sequence: its position and every layer's state."""

    def __init__(self, model):
        self.pos = 0
        self.state = [{} for _ in model.c["layers"]]


def parallel_layer(x, W, l, L, eps, st, p0):
    """Timerax: x += mixer(norm(x)) + ff(norm(x)), one norm for both"""
    h, pre = one_plus_norm(x, W[f"l{l}.norm1"], eps), f"l{l}.mix"
    if L["type"] == "parallel":
        y = parallel_mixer(h, W, pre, L["mixer"], eps, st, p0)
    elif L["type"] == "channel_delta":
        y = channel_delta(h, W, pre, L["mixer"], eps, st)
    else:
        raise ValueError(L["type"])
    if L.get("mlp"):
        y = y + moe(h, W, f"l{l}.mlp", L["mlp"])
    return x + y


def sandwich_layer(x, W, l, L, eps, st, p0):
    """Ranutar: a norm before and behind each sublayer, a causal convolution over time in front of each"""
    p, m = f"l{l}", L["mixer"]
    h = input_conv(one_plus_norm(x, W[p + ".norm1"], eps), W[p + ".canon1"], st.setdefault("conv1", {}))
    s = st.setdefault("mix", {})
    if L["type"] == "wkv":
        y = wkv(h, W, p + ".mix", m, eps, s)
    elif L["type"] == "delta":
        y = head_delta(h, W, p + ".mix", m, eps, s)
    elif L["type"] == "latent_attention":
        y = latent_attention(h, W, p + ".mix", m, eps, s, p0)
    else:
        raise ValueError(L["type"])
    x = x + one_plus_norm(y, W[p + ".norm1b"], eps)
    if L.get("mlp"):
        h = input_conv(one_plus_norm(x, W[p + ".norm2"], eps), W[p + ".canon2"], st.setdefault("conv2", {}))
        y = xielu(h @ W[p + ".mlp.up"].T, *W[p + ".mlp.act"]) @ W[p + ".mlp.down"].T
        x = x + one_plus_norm(y, W[p + ".norm2b"], eps)
    return x


class Model:
    LAYER = {"Timerax": parallel_layer, "Ranutar": sandwich_layer}

    def __init__(self, config, tensors):
        self.c = config
        self.W = {k: np.asarray(v, F) for k, v in tensors.items()}
        self.layer = self.LAYER[config["architecture"]]

    def run(self, seq, tokens, trace=None):
        """logits [tokens, vocab]; trace: a list that gets the residual stream after every layer"""
        c, W, eps = self.c, self.W, self.c["norm"]["eps"]
        x = W["embed"][np.asarray(tokens)]
        for l, L in enumerate(c["layers"]):
            x = self.layer(x, W, l, L, eps, seq.state[l], seq.pos)
            if trace is not None:
                trace.append(x.copy())
        seq.pos += len(tokens)
        z = one_plus_norm(x, W["final.norm"], eps) @ W["head"].T * c.get("logit_scale", 1.0)
        cap = c.get("logit_softcap")
        return cap * np.tanh(z / cap) if cap else z
