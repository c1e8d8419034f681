"""CPU: the Nukizen design's configuration reader and registry, its tensor names and sizes, and properties of the plain
restatement in tests/nukizen_oracle.py that the GPU tests lean on."""
import copy
import math

import numpy as np
import pytest

import nukizen_oracle as O
from nukizen_oracle import att, lru, par

from qwen_inference_engine_amd import _lib
from qwen_inference_engine_amd import spec as S

LAYERS = [lru(), att(size=7), par(heads=6, kv_heads=3, dim=8, vdim=20, rot_dims=0, conv=5), att(size=9, softcap=None, kv_from=1, mlp=None),
          lru(width=20, blocks=1, conv=1, mlp=None)]


def test_config_reader_and_registry():
    sp = S.spec_from_config(O.config(LAYERS, vocab=77, width=24, logit_softcap=12.5))
    assert isinstance(sp, S.LayeredSpec) and "Nukizen" in S.ARCHITECTURES
    assert (sp.block, sp.shared_norm, sp.tied_head, sp.logit_softcap, sp.loop) == ("parallel", True, False, 12.5, None)
    r, a, p, b, r1 = (L.mixer for L in sp.layers)
    assert isinstance(r, S.RgLru) and (r.width, r.blocks, r.conv, r.decay) == (36, 3, 4, 8.0)
    assert (a.mask, a.mask_size, a.softcap, a.head_gate, a.kv_from, a.qk_norm) == ("chunk", 7, 9.0, True, None, "none")
    assert (b.mask_size, b.softcap, b.kv_from) == (9, 0.0, 1) and sp.layers[3].mlp is None and (r1.conv, r1.blocks) == (1, 1)
    assert isinstance(p, S.AttentionWithRecurrence) and isinstance(p.rec, S.GatedDelta) and p.normed and p.attn_scale == p.rec_scale == 0.5
    assert (p.attn.qk_norm, p.attn.sink, p.attn.rot_dims, p.attn.head_gate) == ("row", True, 0, False)
    y = S.spec_from_config(O.config([par()])).layers[0].mixer.attn
    assert y.rot_scaling == (5.0, 0.4, 3.0, 24.0) and y.rot_scaling_kind == "yarn"
    assert S.spec_from_config(O.config([par()], logit_softcap=None)).logit_softcap == 0.0
    arch, _keep = sp.to_c()
    assert arch.block == _lib.QIE_BLOCK_PARALLEL and arch.shared_norm == 1 and arch.logit_softcap == 12.5
    assert [arch.layers[i].kv_from for i in range(5)] == [-1, -1, -1, 1, -1]
    assert arch.layers[0].rglru.blocks == 3 and arch.layers[2].rec.kind == _lib.QIE_REC_DELTA and arch.layers[2].delta.conv == 5
    assert arch.layers[2].mix_norm == 1 and arch.layers[1].ff_act == _lib.QIE_ACT_RELU_GATED


def test_tensor_names_and_sizes():
    cfg = O.config(LAYERS, vocab=77, width=24)
    shapes = {k: list(v.shape) for k, v in O.random_weights(cfg).items()}
    sp = S.spec_from_config(cfg)
    assert sp.tensor_shapes() == shapes
    assert "l3.mix.k" not in shapes and "l0.norm2" not in shapes and "head" in shapes
    assert sp.cache_row_elems() == 2 * (16 + 12) + 3 * (8 + 20)          # layer 3 keeps no rows of its own
    assert sp.state_elems() == 36 * 4 + (4 * 10 * 14 + 4 * (2 * 2 * 10 + 4 * 14)) + 20


@pytest.mark.parametrize("change", [
    lambda c: c["layers"][0].update(type="lru"), lambda c: c["layers"][1]["mlp"].update(kind="moe"),
    lambda c: c["layers"][0]["mixer"].update(blocks=5), lambda c: c["layers"][3]["mixer"].update(kv_from=3),
    lambda c: c["layers"][3]["mixer"].update(kv_from=0), lambda c: c["layers"][3]["mixer"].update(dim=8),
    lambda c: c["layers"][1]["mixer"]["rot"].update(scaling={"factor": 0.0, "original": 24, "fast": 3.0, "slow": 1.0})])
def test_refusals(change):
    cfg = copy.deepcopy(O.config(LAYERS))
    change(cfg)
    with pytest.raises(ValueError):
        S.spec_from_config(cfg)


# ------------------------------------------------------------------ the restatement's own properties
def test_blocks_of_positions():
    v = O.same_block(9, 4)
    assert [list(np.flatnonzero(v[i])) for i in (0, 3, 4, 7, 8)] == [[0], [0, 1, 2, 3], [4], [4, 5, 6, 7], [8]]
    assert O.same_block(5, 1).sum() == 5 and O.same_block(5, 9).sum() == 15


def test_yarn_frequencies_keep_the_fast_pairs_and_slow_the_last():
    rot = {"dims": 16, "base": 500.0, "scaling": {"factor": 5.0, "original": 24, "fast": 3.0, "slow": 0.4}}
    f, amp = O.frequencies(rot)
    g, one = O.frequencies({"dims": 16, "base": 500.0})
    assert one == 1.0 and np.isclose(amp, 0.1 * math.log(5.0) + 1.0)
    assert f[0] == g[0] and np.isclose(f[-1], g[-1] / 5.0) and ((g / 5.0 <= f + 1e-15) & (f <= g)).all()
    assert ((f < g - 1e-12) & (f > g / 5.0 + 1e-12)).any()                   # and a blend between the two
    x = np.ones((30, 1, 20))
    y = O.rotate(x, rot)
    assert np.allclose(y[:, :, 16:], 1.0) and np.allclose((y[..., :16] ** 2).sum(-1), 16 * amp ** 2)


def test_soft_bound():
    z = np.array([-1e3, -0.01, 0.0, 0.01, 1e3])
    assert np.allclose(O.cap(z, 5.0), [-5, -0.01, 0, 0.01, 5], atol=1e-6) and O.cap(z, None) is z


def test_sink_takes_weight_once_and_unscaled():
    s, mask = np.array([[[0.3, -9e9], [1.0, 2.0]]]), np.tril(np.ones((2, 2), bool))
    w = O.softmax_rows(s, mask, np.array([0.7]))
    assert np.isclose(w[0, 0, 0], math.exp(0.3) / (math.exp(0.3) + math.exp(0.7)))
    assert np.isclose(w[0, 1].sum(), 1 - math.exp(0.7) / (math.exp(1) + math.exp(2) + math.exp(0.7)))


def test_recurrences_equal_their_unrolled_forms():
    cfg = O.config([lru(width=6, blocks=2, conv=2, mlp=None)], width=16)
    W, p = {k: O.f64(v) for k, v in O.random_weights(cfg).items()}, "l0.mix."
    h = np.random.default_rng(1).normal(size=(9, 16))
    x = h @ W[p + "x"].T + W[p + "x.b"]
    prev = np.vstack([np.zeros(6), x[:-1]])                                   # the bias is no input before the start
    u = W[p + "conv"][:, 0] * prev + W[p + "conv"][:, 1] * x + W[p + "conv.b"]
    full = lambda g: np.kron(np.eye(2), np.ones((3, 3))) * np.block([[W[p + g][0], W[p + g][0]], [W[p + g][1], W[p + g][1]]])
    r, i = O.sigmoid(u @ full("ra").T + W[p + "ra.b"].ravel()), O.sigmoid(u @ full("ri").T + W[p + "ri.b"].ravel())
    la = -8 * r * np.log1p(np.exp(W[p + "lam"]))
    S = np.array([sum(np.exp(la[s + 1:t + 1].sum(0)) * np.sqrt(1 - np.exp(2 * la[s])) * i[s] * u[s] for s in range(t + 1)) for t in range(9)])
    want = (S * O.gelu_tanh(h @ W[p + "y"].T + W[p + "y.b"])) @ W[p + "o"].T
    assert np.allclose(O.gated_lru(cfg["layers"][0]["mixer"], W, p, h), want)

    cfg = O.config([par(d_heads=2, d_kv_heads=1, d_dim=4, d_vdim=3, conv=1, mlp=None)], width=16)
    W, p, m = {k: O.f64(v) for k, v in O.random_weights(cfg).items()}, "l0.mix.right.", cfg["layers"][0]["mixer"]["right"]
    q, k, v = (O.silu(h @ W[p + n].T * W[p + n + ".conv"][:, 0]) for n in "qkv")
    unit = lambda z: z / np.sqrt((z * z).sum(-1, keepdims=True) + 1e-6)
    q, k, v = unit(q) / 2, unit(k), v.reshape(9, 2, 3)
    beta, g = O.sigmoid(h @ W[p + "b"].T), np.exp(-np.exp(W[p + "A_log"]) * O.softplus(h @ W[p + "a"].T + W[p + "dt_bias"]))
    o = np.zeros((9, 2, 3))
    for a in range(2):
        S = np.zeros((4, 3))
        for t in range(9):                                                   # as one linear map per row
            S = (np.eye(4) - beta[t, a] * np.outer(k[t], k[t])) @ (g[t, a] * S) + beta[t, a] * np.outer(k[t], v[t, a])
            o[t, a] = S.T @ q[t]
    want = (O.norm(o, W[p + "norm"], 1e-5).reshape(9, 6) * O.silu(h @ W[p + "g"].T)) @ W[p + "o"].T
    assert np.allclose(O.delta_rule(m, W, p, h, 1e-5), want)


def test_block_reads_one_norm_and_shared_keys_are_the_owners():
    cfg = O.config([att(size=5), att(size=4, kv_from=0, softcap=None, mlp=None)])
    W = {k: O.f64(v) for k, v in O.random_weights(cfg).items()}
    lay, toks = [], [3, 9, 4, 4, 7, 1]
    O.forward(cfg, W, toks, lay)
    x, m = W["embed"][toks], [L["mixer"] for L in cfg["layers"]]
    h = O.norm(x, W["l0.norm1"], 1e-5)
    kv = O.keys_values(m[0], W, "l0.mix.", h, 1e-5, False)
    assert np.allclose(lay[0], x + O.attend(m[0], W, "l0.mix.", h, kv, 1e-5, head_gate=True) + O.relu_ff(W, "l0.mlp.", h))
    h1 = O.norm(lay[0], W["l1.norm1"], 1e-5)
    assert np.allclose(lay[1], lay[0] + O.attend(m[1], W, "l1.mix.", h1, kv, 1e-5, head_gate=True))


def test_joined_branches_have_unit_scale_each():
    a, b = np.array([[3.0, -1.0]]), np.array([[100.0, 100.0]])
    assert np.allclose(O.joined(a, b, [1.0, 2.0], [0.5, 1.0], 0.0), 0.5 * (a / math.sqrt(5) * [1, 2] + np.array([[0.5, 1.0]])))
