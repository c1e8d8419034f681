"""The Nukizen design restated in numpy float64, one function per mechanism.

Slow and plain on purpose: whole sequences at once, explicit loops over positions where a recurrence runs, no cache
and no batching.  Shares no code with the engine.  ``cfg`` is a config dictionary in the layout of a Nukizen
config.json, ``W`` maps tensor names to arrays.

Notation: T tokens, h the input of a mixer or feed-forward (a normed residual row).
"""
from __future__ import annotations

import math

import numpy as np


def f64(a):
    return np.asarray(a, dtype=np.float64)


def rms_unit(x, eps):
    """x over its root mean square, eps inside the root."""
    return x / np.sqrt(np.mean(x * x, axis=-1, keepdims=True) + eps)


def norm(x, w, eps):
    return rms_unit(x, eps) * f64(w)


def sigmoid(z):
    return np.exp(-np.logaddexp(0.0, -f64(z)))


def silu(z):
    return z * sigmoid(z)


def softplus(z):
    return np.logaddexp(0.0, f64(z))


def gelu_tanh(z):
    return 0.5 * z * (1.0 + np.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def cap(z, c):
    """Soft bound: near the identity for |z| << c, never beyond +-c.  c None: no bound."""
    return z if c is None else c * np.tanh(z / c)


def causal_conv(x, w, b=None):
    """x [T, C], w [C, taps], b [C] or None: out_t = b + sum_j w[:, j] x_(t - taps + 1 + j); zeros before the start."""
    x, w = f64(x), f64(w)
    T, taps = x.shape[0], w.shape[1]
    out = np.zeros(x.shape) if b is None else np.tile(f64(b), (T, 1))
    for t in range(T):
        for j in range(taps):
            s = t - (taps - 1) + j
            if s >= 0:
                out[t] += w[:, j] * x[s]
    return out


def frequencies(rot):
    """(frequency of every rotated pair, factor on cos and sin) of a rotation: base^(-2i / dims), with YaRN's blend of
    kept and slowed frequencies when the rotation is scaled."""
    dims, base = int(rot["dims"]), float(rot["base"])
    f = np.array([base ** (-2.0 * i / dims) for i in range(dims // 2)])
    sc = rot.get("scaling")
    if not sc:
        return f, 1.0
    factor, original = float(sc["factor"]), float(sc["original"])

    def index_of(turns):   # the (real-valued) pair index that turns this often over the original length
        return dims * math.log(original / (2.0 * math.pi * turns)) / (2.0 * math.log(base))

    lo = max(math.floor(index_of(float(sc["fast"]))), 0)
    hi = min(math.ceil(index_of(float(sc["slow"]))), dims - 1)
    out = []
    for i in range(dims // 2):
        ramp = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(f[i] / factor * ramp + f[i] * (1.0 - ramp))
    return np.array(out), 0.1 * math.log(factor) + 1.0


def rotate(x, rot):
    """x [T, heads, D]: coordinate i < dims / 2 pairs with i + dims / 2, turned by t * f_i; the rest passes."""
    if not rot or int(rot["dims"]) == 0:
        return x
    T, dims = x.shape[0], int(rot["dims"])
    half = dims // 2
    f, amp = frequencies(rot)
    ang = np.arange(T)[:, None] * f[None, :]
    c, s = amp * np.cos(ang)[:, None, :], amp * np.sin(ang)[:, None, :]
    out = x.copy()
    u, v = x[..., :half], x[..., half:dims]
    out[..., :half] = u * c - v * s
    out[..., half:dims] = v * c + u * s
    return out


def same_block(T, size):
    """[T, T] mask: row i sees column j <= i inside its own block of `size` positions."""
    i, j = np.arange(T)[:, None], np.arange(T)[None, :]
    return (j <= i) & (i // size == j // size)


def softmax_rows(scores, mask, sink=None):
    """scores [heads, T, T]; sink [heads] or None: one more term exp(sink_h) in every denominator."""
    s = np.where(mask[None], scores, -np.inf)
    top = s.max(axis=-1, keepdims=True)
    if sink is not None:
        top = np.maximum(top, f64(sink)[:, None, None])
    e = np.exp(s - top)
    den = e.sum(axis=-1, keepdims=True)
    if sink is not None:
        den = den + np.exp(f64(sink)[:, None, None] - top)
    return e / den


def keys_values(m, W, p, h, eps, row_norm):
    """Rotated keys [T, G, D] and values [T, G, Dv] of an attention."""
    G, D, Dv, T = int(m["kv_heads"]), int(m["dim"]), int(m["vdim"]), h.shape[0]
    k = h @ f64(W[p + "k"]).T
    if row_norm:
        k = norm(k, W[p + "k.norm"], eps)
    return rotate(k.reshape(T, G, D), m.get("rot")), (h @ f64(W[p + "v"]).T).reshape(T, G, Dv)


def attend(m, W, p, h, kv, eps, row_norm=False, sink=False, head_gate=False):
    """Grouped-query attention inside blocks of positions.  row_norm: q is normed as one row before it is split into
    heads; sink: a learned term per head in the denominator; head_gate: a sigmoid per head on the outputs."""
    H, G, D, Dv, T = int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"]), h.shape[0]
    q = h @ f64(W[p + "q"]).T
    if row_norm:
        q = norm(q, W[p + "q.norm"], eps)
    q = rotate(q.reshape(T, H, D), m.get("rot"))
    k, v = kv
    rep = H // G
    scores = np.stack([q[:, a] @ k[:, a // rep].T for a in range(H)]) * float(m["scale"])
    scores = cap(scores, m.get("softcap"))
    wts = softmax_rows(scores, same_block(T, int(m["mask"]["size"])), W[p + "sink"] if sink else None)
    o = np.stack([wts[a] @ v[:, a // rep] for a in range(H)], axis=1)
    if head_gate:
        o = o * sigmoid(h @ f64(W[p + "g"]).T)[:, :, None]
    return o.reshape(T, H * Dv) @ f64(W[p + "o"]).T


def delta_rule(m, W, p, h, eps):
    """Gated delta rule: S <- g S; u = beta (v - S^T k); S <- S + k u^T; o = S^T q, g and beta one number per head."""
    H, G, D, Dv, T = int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"]), h.shape[0]
    q, k, v = (silu(causal_conv(h @ f64(W[p + n]).T, W[p + n + ".conv"])) for n in "qkv")
    q, k, v = q.reshape(T, G, D), k.reshape(T, G, D), v.reshape(T, H, Dv)
    q = q / np.sqrt((q * q).sum(-1, keepdims=True) + 1e-6) * D ** -0.5
    k = k / np.sqrt((k * k).sum(-1, keepdims=True) + 1e-6)
    beta = sigmoid(h @ f64(W[p + "b"]).T)
    g = np.exp(-np.exp(f64(W[p + "A_log"])) * softplus(h @ f64(W[p + "a"]).T + f64(W[p + "dt_bias"])))
    o = np.zeros((T, H, Dv))
    for a in range(H):
        S, kh = np.zeros((D, Dv)), a // (H // G)
        for t in range(T):
            S = g[t, a] * S
            u = beta[t, a] * (v[t, a] - S.T @ k[t, kh])
            S = S + np.outer(k[t, kh], u)
            o[t, a] = S.T @ q[t, kh]
    o = norm(o, W[p + "norm"], eps).reshape(T, H * Dv)
    return (o * silu(h @ f64(W[p + "g"]).T)) @ f64(W[p + "o"]).T


def gated_lru(m, W, p, h):
    """Real-gated linear recurrence per channel behind a short convolution, times a gelu branch."""
    n, nb, T = int(m["width"]), int(m["blocks"]), h.shape[0]
    bs = n // nb
    y = gelu_tanh(h @ f64(W[p + "y"]).T + f64(W[p + "y.b"]))
    u = causal_conv(h @ f64(W[p + "x"]).T + f64(W[p + "x.b"]), W[p + "conv"], W[p + "conv.b"])
    r, i = np.zeros((T, n)), np.zeros((T, n))
    for b in range(nb):
        c = slice(b * bs, (b + 1) * bs)
        r[:, c] = sigmoid(u[:, c] @ f64(W[p + "ra"])[b].T + f64(W[p + "ra.b"])[b])
        i[:, c] = sigmoid(u[:, c] @ f64(W[p + "ri"])[b].T + f64(W[p + "ri.b"])[b])
    log_a = -8.0 * r * softplus(W[p + "lam"])
    S, out = np.zeros(n), np.zeros((T, n))
    for t in range(T):
        S = np.exp(log_a[t]) * S + np.sqrt(-np.expm1(2.0 * log_a[t])) * i[t] * u[t]
        out[t] = S * y[t]
    return out @ f64(W[p + "o"]).T


def relu_ff(W, p, h):
    return (np.maximum(h @ f64(W[p + "gate"]).T, 0.0) * (h @ f64(W[p + "up"]).T)) @ f64(W[p + "down"]).T


def joined(a, b, wa, wb, eps):
    """Half the sum of two branches, each normed over the model width with its own weights."""
    return 0.5 * (norm(a, wa, eps) + norm(b, wb, eps))


def forward(cfg, W, tokens, layers_out=None):
    """Logits [T, vocab] of one sequence.  layers_out (a list) receives the stream after every layer."""
    eps = float(cfg["norm"]["eps"])
    x = f64(W["embed"])[np.asarray(tokens)]
    kept = {}   # layer -> its keys and values
    for i, L in enumerate(cfg["layers"]):
        m, p = L["mixer"], f"l{i}.mix."
        h = norm(x, W[f"l{i}.norm1"], eps)
        if L["type"] == "rglru":
            y = gated_lru(m, W, p, h)
        elif L["type"] == "attention":
            j = m.get("kv_from")
            if j is None:
                kept[i] = keys_values(m, W, p, h, eps, False)
            y = attend(m, W, p, h, kept[i if j is None else int(j)], eps, head_gate=True)
        elif L["type"] == "parallel":
            pl, pr = p + "left.", p + "right."
            kept[i] = keys_values(m["left"], W, pl, h, eps, True)
            left = attend(m["left"], W, pl, h, kept[i], eps, row_norm=True, sink=True)
            y = joined(left, delta_rule(m["right"], W, pr, h, eps), W[pl + "out"], W[pr + "out"], eps)
        else:
            raise ValueError(L["type"])
        if L.get("mlp") is not None:
            y = y + relu_ff(W, f"l{i}.mlp.", h)
        x = x + y
        if layers_out is not None:
            layers_out.append(x.copy())
    return cap(norm(x, W["final.norm"], eps) @ f64(W["head"]).T, cfg.get("logit_softcap"))


# ---------------------------------------------------------------- small configurations and random weights
def dense(ff=40):
    return {"kind": "dense", "ff": ff}


def _mlp(mlp):
    return dense() if mlp == "dense" else mlp


def lru(width=36, blocks=3, conv=4, mlp="dense"):
    return {"type": "rglru", "mixer": {"width": width, "blocks": blocks, "conv": conv}, "mlp": _mlp(mlp)}


def _attention(heads, kv_heads, dim, vdim, size, rot_dims, base, scale, scaling):
    a = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "mask": {"size": size},
         "scale": scale if scale is not None else dim ** -0.5}
    if rot_dims:
        a["rot"] = {"base": base, "dims": rot_dims}
        if scaling:
            a["rot"]["scaling"] = dict(zip(("factor", "original", "fast", "slow"), scaling))
    return a


def att(heads=4, kv_heads=2, dim=16, vdim=12, size=11, rot_dims=8, base=10000.0, scale=None, scaling=None, softcap=9.0, kv_from=None,
        mlp="dense"):
    m = _attention(heads, kv_heads, dim, vdim, size, rot_dims, base, scale, scaling)
    if softcap:
        m["softcap"] = softcap
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "attention", "mixer": m, "mlp": _mlp(mlp)}


YARN = (5.0, 24, 3.0, 0.4)   # factor, original length, fast and slow turns


def par(heads=4, kv_heads=2, dim=16, vdim=12, size=13, rot_dims=16, base=500.0, scale=None, scaling=YARN, d_heads=4, d_kv_heads=2, d_dim=10,
        d_vdim=14, conv=3, mlp="dense"):
    return {"type": "parallel", "mlp": _mlp(mlp), "mixer": {
        "left": _attention(heads, kv_heads, dim, vdim, size, rot_dims, base, scale, scaling),
        "right": {"heads": d_heads, "kv_heads": d_kv_heads, "dim": d_dim, "vdim": d_vdim, "conv": conv}}}


def config(layers, vocab=101, width=40, eps=1e-5, logit_softcap=6.0):
    cfg = {"architecture": "Nukizen", "vocab": vocab, "width": width, "norm": {"eps": eps}, "layers": layers}
    if logit_softcap:
        cfg["logit_softcap"] = logit_softcap
    return cfg


def to_bf16_exact(a):
    """float32 values rounded to the nearest bf16 (kept as float32)."""
    u = np.ascontiguousarray(a, dtype=np.float32).view(np.uint32)
    u = (u + 0x7FFF + ((u >> 16) & 1)) & np.uint32(0xFFFF0000)
    return u.view(np.float32).reshape(np.shape(a))


def random_weights(cfg, seed=0, qk_gain=2.0):
    """{name: float32 array of exact bf16 values}.  The branches' output projections are small beside the residual rows,
    so that a rounding error shrinks from layer to layer.  qk_gain: how sharp the softmaxes are."""
    rng = np.random.default_rng(seed)
    W, V, T = cfg["width"], cfg["vocab"], {}

    def lin(o, i, gain=1.0):
        return rng.normal(0.0, gain / math.sqrt(i), (o, i))

    def vec(n, sd=0.2, mean=0.0):
        return mean + rng.normal(0.0, sd, n)

    def attention(x, a, own=True, row_norm=False):
        H, G, D, Dv = a["heads"], a["kv_heads"], a["dim"], a["vdim"]
        T[x + "q"], T[x + "o"] = lin(H * D, W, qk_gain), lin(W, H * Dv, 0.5)
        if own:
            T[x + "k"], T[x + "v"] = lin(G * D, W, qk_gain), lin(G * Dv, W)
        if row_norm:
            T[x + "q.norm"], T[x + "k.norm"] = vec(H * D, 0.4, qk_gain), vec(G * D, 0.4, 1.0)
            T[x + "sink"], T[x + "out"] = vec(H, 1.0, 1.0), vec(W, 0.2, 0.9)

    T["embed"], T["final.norm"], T["head"] = rng.normal(0, 1.0, (V, W)), vec(W, 0.2, 1.0), lin(V, W, 2.5)
    for i, L in enumerate(cfg["layers"]):
        p, m = f"l{i}.", L["mixer"]
        T[p + "norm1"] = vec(W, 0.25, 1.0)
        x = p + "mix."
        if L["type"] == "rglru":
            n, nb, bs = m["width"], m["blocks"], m["width"] // m["blocks"]
            T[x + "y"], T[x + "y.b"], T[x + "x"], T[x + "x.b"] = lin(n, W, 1.5), vec(n, 0.5), lin(n, W), vec(n, 0.5)
            T[x + "conv"], T[x + "conv.b"] = rng.normal(0, 0.6, (n, m["conv"])), vec(n, 0.3)
            for g in ("ra", "ri"):
                T[x + g] = rng.normal(0, 1.5 / math.sqrt(bs), (nb, bs, bs))
                T[x + g + ".b"] = rng.normal(0, 0.7, (nb, bs))
            T[x + "lam"], T[x + "o"] = vec(n, 1.0, -2.0), lin(W, n, 0.5)
        elif L["type"] == "attention":
            attention(x, m, own=m.get("kv_from") is None)
            T[x + "g"] = lin(m["heads"], W, 1.5)
        else:
            attention(x + "left.", m["left"], row_norm=True)
            c, x = m["right"], x + "right."
            nk, nv, H = c["kv_heads"] * c["dim"], c["heads"] * c["vdim"], c["heads"]
            for n, k in (("q", nk), ("k", nk), ("v", nv)):
                T[x + n], T[x + n + ".conv"] = lin(k, W, 1.5), rng.normal(0, 0.7, (k, c["conv"]))
            T[x + "b"], T[x + "a"], T[x + "g"] = lin(H, W, 1.5), lin(H, W), lin(nv, W)
            T[x + "A_log"], T[x + "dt_bias"], T[x + "norm"] = vec(H, 0.7, -1.0), vec(H, 0.7, -1.0), vec(c["vdim"], 0.2, 1.0)
            T[x + "o"], T[x + "out"] = lin(W, nv, 0.5), vec(W, 0.2, 0.9)
        if L.get("mlp") is not None:
            ff = L["mlp"]["ff"]
            T[p + "mlp.gate"], T[p + "mlp.up"], T[p + "mlp.down"] = lin(ff, W, 1.5), lin(ff, W), lin(W, ff, 0.4)
    return {k: to_bf16_exact(v) for k, v in T.items()}
