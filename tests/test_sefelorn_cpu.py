"""CPU: the Sefelorn design's configuration reader and registry, its tensor names and sizes, and properties of the plain
restatement in tests/sefelorn_oracle.py that the GPU tests lean on."""
import copy

import numpy as np
import pytest

import sefelorn_oracle as O
from sefelorn_oracle import dense, par, ssm

from qwen_inference_engine_amd import _lib
from qwen_inference_engine_amd import spec as S


def public(cfg):
    return {k: v for k, v in cfg.items() if not k.startswith("_")}


LAYERS = [ssm(), par(), par(heads=6, kv_heads=3, dim=8, vdim=20, keep=0, rot_dims=0, rank=3, mlp=None), ssm(mlp=None)]


def test_config_reader_and_registry():
    sp = S.spec_from_config(public(O.config(LAYERS, vocab=77, width=24, embed_scale=2.5, logit_scale=0.3, loop=(1, 3, 2))))
    assert isinstance(sp, S.LayeredSpec) and "Sefelorn" in S.ARCHITECTURES
    assert (sp.block, sp.tied_head, sp.embed_scale, sp.logit_scale, sp.loop) == ("parallel", True, 2.5, 0.3, (1, 3, 2))
    assert sp.runs() == [0, 1, 2, 1, 2, 3]
    s, p, q = sp.layers[0].mixer, sp.layers[1].mixer, sp.layers[2].mixer
    assert isinstance(s, S.StateSpace) and (s.inner, s.conv_channels) == (48, 48 + 2 * 2 * 10)
    assert isinstance(p, S.AttentionWithRecurrence) and isinstance(p.rec, S.KeyDecayRecurrence) and p.rec.rank == 0
    assert (p.attn_scale, p.rec_scale, p.rec.tau) == (0.9, 1.15, 4.0)
    a = p.attn
    assert a.qk_bias and a.v_bias and (a.mask, a.mask_size, a.mask_keep) == ("window", 11, 3) and (a.rot_dims, a.rot_layout) == (8, "halves")
    assert (q.attn.rot_dims, q.attn.mask_keep) == (0, 0) and sp.layers[2].mlp is None
    assert (sp.layers[0].mlp.act, sp.layers[0].mlp.limit) == ("clamped_gated", 1.25)
    arch, _keep = sp.to_c()
    assert arch.block == _lib.QIE_BLOCK_PARALLEL and abs(arch.logit_scale - 0.3) < 1e-7 and arch.loop_times == 2
    assert arch.layers[0].ssm.state == 10 and arch.layers[1].gqa.mask_keep == 3 and arch.layers[1].rec.kind == _lib.QIE_REC_KEY_DECAY


def test_tensor_names_and_sizes_from_the_tensors():
    cfg = O.config(LAYERS, vocab=77, width=24)
    T = O.random_weights(cfg)
    shapes_in = {k: list(v.shape) for k, v in T.items()}
    sp = S.with_tensor_sizes(S.spec_from_config(public(cfg)), shapes_in)
    assert (sp.layers[1].mixer.rec.rank, sp.layers[2].mixer.rec.rank) == (5, 3)
    assert sp.tensor_shapes() == shapes_in
    assert "head" not in shapes_in and "l3.norm2" not in shapes_in
    assert sp.cache_row_elems() == 2 * (16 + 12) + 3 * (8 + 20)
    assert sp.state_elems() == 2 * (4 * 10 * 12 + 2 * 88) + 2 * 3 * 10 * 14
    with pytest.raises(ValueError):
        S.with_tensor_sizes(S.spec_from_config(public(cfg)), {})


@pytest.mark.parametrize("change", [
    lambda c: c["layers"][0].update(type="mamba"), lambda c: c["layers"][1]["mlp"].update(kind="moe"),
    lambda c: c["layers"][0]["mixer"].update(groups=3), lambda c: c["layers"][0]["mixer"].update(norm_groups=5),
    lambda c: c.update(loop={"start": 2, "stop": 9, "times": 2}), lambda c: c.update(loop={"start": 0, "stop": 1, "times": 0})])
def test_refusals(change):
    cfg = copy.deepcopy(public(O.config(LAYERS)))
    change(cfg)
    with pytest.raises(ValueError):
        S.spec_from_config(cfg)


# ------------------------------------------------------------------ the restatement's own properties
def test_window_keeps_the_first_tokens():
    v = O.visible(12, 4, 2)
    assert [list(np.flatnonzero(v[i])) for i in (0, 3, 5, 6, 11)] == [[0], [0, 1, 2, 3], [0, 1, 2, 3, 4, 5], [0, 1, 3, 4, 5, 6],
                                                                   [0, 1, 8, 9, 10, 11]]
    assert not O.visible(12, 4, 0)[11, :8].any() and O.visible(5, 1, 9).sum() == 15      # all of them kept: causal


def test_rotation_is_relative_and_partial():
    rng = np.random.default_rng(0)
    q, k = rng.normal(size=(1, 10)), rng.normal(size=(1, 10))
    rows = lambda x: O.rotate_halves(np.repeat(x[:, None], 9, axis=0).reshape(9, 1, 10), 6, 50.0)
    a, b = rows(q)[:, 0], rows(k)[:, 0]
    assert np.allclose(a[:, 6:], q[:, 6:]) and np.allclose([a[i + 3] @ b[i] for i in range(6)], a[3] @ b[0])


def test_recurrences_equal_their_unrolled_sums_and_carry_the_first_token():
    cfg = O.config([par(left=0.0, rec_heads=1, rec_dim=4, rec_vdim=3, rank=2, mlp=None)], width=16)
    W, p = {k: O.f64(v) for k, v in O.random_weights(cfg).items()}, "l0.mix.right."
    h = np.random.default_rng(1).normal(size=(11, 16))
    m = cfg["layers"][0]["mixer"]["right"]
    q, k, v = h @ W[p + "q"].T * 0.5, h @ W[p + "k"].T, h @ W[p + "v"].T
    al = O.sigmoid(h @ W[p + "a1"].T @ W[p + "a2"].T + W[p + "a2.b"]) ** (1 / 4.0)
    o = np.array([sum((q[t] * k[s] * np.prod(al[s + 1:t + 1], axis=0)).sum() * v[s] for s in range(t + 1)) for t in range(11)])
    want = (O.rms_unit(o, 1e-5) * W[p + "norm"] * O.silu(h @ W[p + "g"].T)) @ W[p + "o"].T
    assert np.allclose(O.key_decay_attention(m, W, p, h, 1e-5), want)

    cfg = O.config([ssm(heads=2, vdim=3, state=4, groups=1, conv=2, norm_groups=2, mlp=None)], width=16)
    W, p, m = {k: O.f64(v) for k, v in O.random_weights(cfg).items()}, "l0.mix.", cfg["layers"][0]["mixer"]
    proj = h @ W[p + "in"].T
    z, xbc, dt = proj[:, :6], proj[:, 6:20], O.softplus(proj[:, 20:] + W[p + "dt_bias"])
    prev = np.vstack([np.zeros(14), xbc[:-1]])
    xbc = O.silu(W[p + "conv"][:, 0] * prev + W[p + "conv"][:, 1] * xbc + W[p + "conv.b"])
    x, B, C = xbc[:, :6].reshape(11, 2, 3), xbc[:, 6:10], xbc[:, 10:]
    la = -np.exp(W[p + "A_log"]) * dt
    y = np.array([[sum(np.exp(la[s + 1:t + 1, a].sum()) * dt[s, a] * (C[t] @ B[s]) * x[s, a] for s in range(t + 1)) + W[p + "D"][a] * x[t, a]
                   for a in range(2)] for t in range(11)]).reshape(11, 6) * O.silu(z)
    y = np.concatenate([O.rms_unit(y[:, :3], 1e-5), O.rms_unit(y[:, 3:], 1e-5)], axis=1) * W[p + "norm"]
    assert np.allclose(O.state_space(m, W, p, h, 1e-5), y @ W[p + "o"].T)


def test_clamped_feed_forward_values():
    W = {"gate": np.array([[1.0]]), "up": np.array([[2.0]]), "down": np.array([[1.0]])}
    f = lambda x: O.clamped_ff({"limit": 1.5}, W, "", np.array([[x]]))[0, 0]
    g = lambda z: z / (1 + np.exp(-1.702 * z))
    assert np.isclose(f(0.5), g(0.5) * 2.0) and np.isclose(f(9.0), g(1.5) * 2.5) and np.isclose(f(-9.0), g(-9.0) * -0.5)


def test_repeated_group_adds_the_embedding_once_a_pass():
    cfg = O.config([ssm(), par(), ssm(mlp=None)], loop=(1, 3, 3))
    assert O.layer_runs(cfg) == [(0, False), (1, False), (2, False), (1, True), (2, False), (1, True), (2, False)]
    W = {k: np.zeros_like(v) if k.endswith(".o") or k.endswith(".down") else v for k, v in O.random_weights(cfg).items()}
    lay = []
    O.forward(cfg, W, [3, 5], lay)          # branches silenced: only the added embeddings remain
    x0 = O.f64(W["embed"])[[3, 5]] * 3.0
    assert [bool(np.allclose(a, n * x0)) for a, n in zip(lay, (1, 1, 1, 2, 2, 3, 3))] == [True] * 7


def test_parallel_block_branches_read_the_same_row():
    cfg = O.config([ssm()])
    W = {k: O.f64(v) for k, v in O.random_weights(cfg).items()}
    lay = []
    O.forward(cfg, W, [7], lay)
    x0 = W["embed"][[7]] * 3.0
    want = x0 + O.state_space(cfg["layers"][0]["mixer"], W, "l0.mix.", O.norm(x0, W["l0.norm1"], 1e-5), 1e-5) \
        + O.clamped_ff(dense(), W, "l0.mlp.", O.norm(x0, W["l0.norm2"], 1e-5))
    assert np.allclose(lay[0], want)
