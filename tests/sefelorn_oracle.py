"""The Sefelorn design restated in numpy float64, one function per mechanism.

Slow and plain on purpose: whole sequences at once, explicit loops over positions where a recurrence runs, no cache
and no batching.  Shares no code with the engine.  ``cfg`` is a config dictionary in the layout of a Sefelorn
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
    return np.logaddexp(0.0, z)


def causal_conv(x, w, b):
    """x [T, C], w [C, taps], b [C]: out_t = b + sum_j w[:, j] x_(t - taps + 1 + j); zeros before the start."""
    x, w = f64(x), f64(w)
    T, taps = x.shape[0], w.shape[1]
    out = np.tile(f64(b), (T, 1))
    for t in range(T):
        for j in range(taps):
            s = t - (taps - 1) + j
            if s >= 0:
                out[t] += w[:, j] * x[s]
    return out


def rotate_halves(x, dims, base):
    """x [T, heads, D]: coordinate i < dims / 2 pairs with i + dims / 2, turned by t * base^(-2i / dims)."""
    if dims == 0:
        return x
    T, half = x.shape[0], dims // 2
    f = np.array([base ** (-2.0 * i / dims) for i in range(half)])
    ang = np.arange(T)[:, None] * f[None, :]
    c, s = np.cos(ang)[:, None, :], np.sin(ang)[:, None, :]
    out = x.copy()
    u, v = x[..., :half], x[..., half:dims]
    out[..., :half] = u * c - v * s
    out[..., half:dims] = v * c + u * s
    return out


def visible(T, size, keep):
    """[T, T] mask: row i sees column j <= i within the last `size` positions or among the first `keep`."""
    i, j = np.arange(T)[:, None], np.arange(T)[None, :]
    return (j <= i) & ((i - j < size) | (j < keep))


def softmax_rows(scores, mask):
    s = np.where(mask[None], scores, -np.inf)
    e = np.exp(s - s.max(axis=-1, keepdims=True))
    return e / e.sum(axis=-1, keepdims=True)


def window_attention(m, W, p, h):
    """Grouped-query softmax attention with biased projections, a partial rotary and a sliding window that keeps the
    first tokens of the sequence."""
    H, G, D, Dv = int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"])
    T = h.shape[0]
    q = (h @ f64(W[p + "q"]).T + f64(W[p + "q.b"])).reshape(T, H, D)
    k = (h @ f64(W[p + "k"]).T + f64(W[p + "k.b"])).reshape(T, G, D)
    v = (h @ f64(W[p + "v"]).T + f64(W[p + "v.b"])).reshape(T, G, Dv)
    rot = m.get("rot") or {"dims": 0, "base": 1.0}
    q = rotate_halves(q, int(rot["dims"]), float(rot["base"]))
    k = rotate_halves(k, int(rot["dims"]), float(rot["base"]))
    rep = H // G
    scores = np.stack([q[:, a] @ k[:, a // rep].T for a in range(H)]) * float(m["scale"])
    wts = softmax_rows(scores, visible(T, int(m["mask"]["size"]), int(m["mask"]["keep_first"])))
    o = np.stack([wts[a] @ v[:, a // rep] for a in range(H)], axis=1)
    return o.reshape(T, H * Dv) @ f64(W[p + "o"]).T


def key_decay_attention(m, W, p, h, eps):
    """Gated linear attention: S <- diag(alpha) S + k v^T, o = S^T q; alpha per head and key channel."""
    H, D, Dv, tau = int(m["heads"]), int(m["dim"]), int(m["vdim"]), float(m["tau"])
    T = h.shape[0]
    q = (h @ f64(W[p + "q"]).T).reshape(T, H, D) * D ** -0.5
    k = (h @ f64(W[p + "k"]).T).reshape(T, H, D)
    v = (h @ f64(W[p + "v"]).T).reshape(T, H, Dv)
    z = (h @ f64(W[p + "a1"]).T) @ f64(W[p + "a2"]).T + f64(W[p + "a2.b"])
    alpha = (sigmoid(z) ** (1.0 / tau)).reshape(T, H, D)
    o = np.zeros((T, H, Dv))
    for a in range(H):
        S = np.zeros((D, Dv))
        for t in range(T):
            S = alpha[t, a][:, None] * S + np.outer(k[t, a], v[t, a])
            o[t, a] = S.T @ q[t, a]
    o = (rms_unit(o, eps) * f64(W[p + "norm"])).reshape(T, H * Dv)
    return (o * silu(h @ f64(W[p + "g"]).T)) @ f64(W[p + "o"]).T


def state_space(m, W, p, h, eps):
    """Mamba-2: a scalar decay per head and token, input and output vectors shared by groups of heads, a skip per
    head, the gate before a norm in equal parts."""
    H, Dv, N, G, parts = (int(m[k]) for k in ("heads", "vdim", "state", "groups", "norm_groups"))
    inner, T = H * Dv, h.shape[0]
    proj = h @ f64(W[p + "in"]).T
    z, xbc, dt = proj[:, :inner], proj[:, inner:2 * inner + 2 * G * N], proj[:, 2 * inner + 2 * G * N:]
    xbc = silu(causal_conv(xbc, W[p + "conv"], W[p + "conv.b"]))
    x = xbc[:, :inner].reshape(T, H, Dv)
    B = xbc[:, inner:inner + G * N].reshape(T, G, N)
    C = xbc[:, inner + G * N:].reshape(T, G, N)
    dt = softplus(dt + f64(W[p + "dt_bias"]))
    a, D = np.exp(f64(W[p + "A_log"])), f64(W[p + "D"])
    y = np.zeros((T, H, Dv))
    for hh in range(H):
        S, g = np.zeros((N, Dv)), hh // (H // G)
        for t in range(T):
            S = np.exp(-a[hh] * dt[t, hh]) * S + dt[t, hh] * np.outer(B[t, g], x[t, hh])
            y[t, hh] = S.T @ C[t, g] + D[hh] * x[t, hh]
    y = y.reshape(T, inner) * silu(z)
    y = rms_unit(y.reshape(T, parts, inner // parts), eps).reshape(T, inner) * f64(W[p + "norm"])
    return y @ f64(W[p + "o"]).T


def clamped_ff(mlp, W, p, h):
    lim = float(mlp["limit"])
    g = np.minimum(h @ f64(W[p + "gate"]).T, lim)
    u = np.clip(h @ f64(W[p + "up"]).T, -lim, lim)
    return (g * sigmoid(1.702 * g) * (u + 1.0)) @ f64(W[p + "down"]).T


def layer_runs(cfg):
    """(layer, embedding added first?) of every layer run in order."""
    n, lp = len(cfg["layers"]), cfg.get("loop")
    if not lp:
        return [(i, False) for i in range(n)]
    a, b, t = int(lp["start"]), int(lp["stop"]), int(lp["times"])
    out = [(i, False) for i in range(a)]
    for k in range(t):
        out += [(i, k > 0 and i == a) for i in range(a, b)]
    return out + [(i, False) for i in range(b, n)]


def forward(cfg, W, tokens, layers_out=None):
    """Logits [T, vocab] of one sequence.  layers_out (a list) receives the stream after every layer run."""
    eps = float(cfg["norm"]["eps"])
    x0 = f64(W["embed"])[np.asarray(tokens)] * float(cfg["embedding"]["scale"])
    x = x0.copy()
    for i, again in layer_runs(cfg):
        L, p = cfg["layers"][i], f"l{i}."
        if again:
            x = x + x0
        m, h = L["mixer"], norm(x, W[p + "norm1"], eps)
        if L["type"] == "mamba2":
            y = state_space(m, W, p + "mix.", h, eps)
        elif L["type"] == "parallel":
            y = float(m["left_scale"]) * window_attention(m["left"], W, p + "mix.left.", h) \
                + float(m["right_scale"]) * key_decay_attention(m["right"], W, p + "mix.right.", h, eps)
        else:
            raise ValueError(L["type"])
        if L.get("mlp") is not None:
            y = y + clamped_ff(L["mlp"], W, p + "mlp.", norm(x, W[p + "norm2"], eps))
        x = x + y
        if layers_out is not None:
            layers_out.append(x.copy())
    return norm(x, W["final.norm"], eps) @ f64(W["embed"]).T * float(cfg["logit_scale"])


# ---------------------------------------------------------------- small configurations and random weights
def dense(ff=40, limit=1.25):
    return {"kind": "dense", "ff": ff, "limit": limit}


def ssm(heads=4, vdim=12, state=10, groups=2, conv=3, norm_groups=2, mlp="dense"):
    return {"type": "mamba2", "mixer": {"heads": heads, "vdim": vdim, "state": state, "groups": groups, "conv": conv,
                                        "norm_groups": norm_groups}, "mlp": dense() if mlp == "dense" else mlp}


def par(heads=4, kv_heads=2, dim=16, vdim=12, size=11, keep=3, rot_dims=8, base=10000.0, scale=None, left=0.9, rec_heads=3,
        rec_dim=10, rec_vdim=14, tau=4.0, rank=5, right=1.15, mlp="dense"):
    """rank: rows of a1 - a size only the tensors carry."""
    a = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "mask": {"size": size, "keep_first": keep},
         "scale": scale if scale is not None else dim ** -0.5}
    if rot_dims:
        a["rot"] = {"base": base, "dims": rot_dims}
    return {"type": "parallel", "mixer": {"left": a, "right": {"heads": rec_heads, "dim": rec_dim, "vdim": rec_vdim, "tau": tau},
                                          "left_scale": left, "right_scale": right},
            "mlp": dense() if mlp == "dense" else mlp, "_rank": rank}


def config(layers, vocab=101, width=40, eps=1e-5, embed_scale=3.0, logit_scale=0.7, loop=None):
    cfg = {"architecture": "Sefelorn", "vocab": vocab, "width": width, "norm": {"eps": eps}, "embedding": {"scale": embed_scale},
           "logit_scale": logit_scale, "layers": [{k: v for k, v in L.items() if k != "_rank"} for L in layers]}
    if loop:
        cfg["loop"] = dict(zip(("start", "stop", "times"), loop))
    cfg["_ranks"] = [L.get("_rank") for L in layers]
    return cfg


def to_bf16_exact(a):
    """float32 values rounded to the nearest bf16 (kept as float32)."""
    u = np.ascontiguousarray(a, dtype=np.float32).view(np.uint32)
    u = (u + 0x7FFF + ((u >> 16) & 1)) & np.uint32(0xFFFF0000)
    return u.view(np.float32).reshape(np.shape(a))


def random_weights(cfg, seed=0, qk_gain=2.0):
    """{name: float32 array of exact bf16 values} for a config made by config().  The branches' output projections are
    small beside the residual rows, so that a rounding error shrinks from layer to layer.  qk_gain: how sharp the
    softmaxes are."""
    rng = np.random.default_rng(seed)
    W, V, T = cfg["width"], cfg["vocab"], {}

    def lin(o, i, gain=1.0):
        return rng.normal(0.0, gain / math.sqrt(i), (o, i))

    def vec(n, sd=0.2, mean=0.0):
        return mean + rng.normal(0.0, sd, n)

    T["embed"], T["final.norm"] = rng.normal(0, 0.4, (V, W)), vec(W, 0.2, 1.0)
    for i, L in enumerate(cfg["layers"]):
        p, m = f"l{i}.", L["mixer"]
        T[p + "norm1"] = vec(W, 0.25, 1.0)
        if L["type"] == "mamba2":
            x, inner = p + "mix.", m["heads"] * m["vdim"]
            C = inner + 2 * m["groups"] * m["state"]
            T[x + "in"], T[x + "conv"], T[x + "conv.b"] = lin(inner + C + m["heads"], W, 1.5), rng.normal(0, 0.6, (C, m["conv"])), vec(C)
            T[x + "dt_bias"], T[x + "A_log"], T[x + "D"] = vec(m["heads"], 1.0, -1.0), vec(m["heads"], 0.7), vec(m["heads"], 0.4, 0.8)
            T[x + "norm"], T[x + "o"] = vec(inner, 0.2, 1.0), lin(W, inner, 0.5)
        else:
            a, c = m["left"], m["right"]
            x, H, G = p + "mix.left.", a["heads"], a["kv_heads"]
            T[x + "q"], T[x + "k"], T[x + "v"] = lin(H * a["dim"], W, qk_gain), lin(G * a["dim"], W, qk_gain), lin(G * a["vdim"], W)
            T[x + "q.b"], T[x + "k.b"], T[x + "v.b"] = vec(H * a["dim"], 0.5), vec(G * a["dim"], 0.5), vec(G * a["vdim"], 0.5)
            T[x + "o"] = lin(W, H * a["vdim"], 0.5)
            x, nk, nv, r = p + "mix.right.", c["heads"] * c["dim"], c["heads"] * c["vdim"], cfg["_ranks"][i]
            T[x + "q"], T[x + "k"], T[x + "v"], T[x + "g"] = lin(nk, W, 1.5), lin(nk, W, 1.5), lin(nv, W), lin(nv, W)
            T[x + "a1"], T[x + "a2"], T[x + "a2.b"], T[x + "norm"] = lin(r, W), lin(nk, r, 2.0), vec(nk, 1.0, 1.0), vec(c["vdim"], 0.2, 1.0)
            T[x + "o"] = lin(W, nv, 0.5)
        if L.get("mlp") is not None:
            ff = L["mlp"]["ff"]
            T[p + "norm2"] = vec(W, 0.25, 1.0)
            T[p + "mlp.gate"], T[p + "mlp.up"], T[p + "mlp.down"] = lin(ff, W, 1.5), lin(ff, W), lin(W, ff, 0.4)
    return {k: to_bf16_exact(v) for k, v in T.items()}
