"""GPU: the Sefelorn design on the layered engine tier (parallel blocks behind two norms, a repeated group, the Mamba-2
state space, a sliding-window attention that keeps the first tokens beside gated linear attention, the clamped gated
feed-forward, the scaled tied head) against the plain numpy restatement in tests/sefelorn_oracle.py, on small random
models of several shapes.

fp32 engines are held to REL32 of the logits' spread, bf16 engines to REL16.  Where random weights would hide a fault
the weights are made to show it: beacon tokens (an id whose key alone stands out for every query) placed at a window's
edge, among the kept first tokens and just behind them, decays near one that keep the first tokens alive in the
recurrent states - and the restatement's own sensitivity to the thing under test is asserted first.
"""
import copy
import json
import os
import subprocess
import sys

import numpy as np
import pytest

import sefelorn_oracle as O
from sefelorn_oracle import dense, par, ssm

pytestmark = pytest.mark.gpu

REL32 = 2e-4
REL16 = 5e-2
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))


def words(a):
    """float32 values that are exact bf16 -> bf16 words"""
    return (np.ascontiguousarray(a, dtype=np.float32).view(np.uint32) >> 16).astype(np.uint16).reshape(np.shape(a))


MIXED = [ssm(), par(), par(heads=6, kv_heads=3, dim=12, vdim=20, size=7, keep=2, rot_dims=12, rec_heads=2, rec_dim=18, rec_vdim=9,
                           tau=11.0, rank=3, mlp=dense(24, 0.5)),
         ssm(heads=6, vdim=7, state=21, groups=1, conv=4, norm_groups=3, mlp=None), par(size=20, keep=0, kv_heads=4, mlp=None)]
LOOP = (1, 4, 2)


class Model:
    def __init__(self, layers, seed=0, vocab=101, width=40, dtype="float32", max_ctx=512, slots=4, page_tokens=16, n_pages=0, eps=1e-5,
                 loop=None, tweak=None, use_graph=True, embed_scale=3.0, logit_scale=0.7):
        import qwen_inference_engine_amd as q
        from qwen_inference_engine_amd.spec import with_tensor_sizes
        self.rng = np.random.default_rng(seed)
        self.cfg = O.config(layers, vocab=vocab, width=width, eps=eps, loop=loop, embed_scale=embed_scale, logit_scale=logit_scale)
        self.T = O.random_weights(self.cfg, seed=seed, qk_gain=2.0 if dtype == "float32" else 1.0)
        if tweak is not None:
            tweak(self.T, self.cfg)
            self.T = {k: O.to_bf16_exact(v) for k, v in self.T.items()}
        public = {k: v for k, v in self.cfg.items() if not k.startswith("_")}
        self.spec = with_tensor_sizes(q.spec_from_config(public), {k: list(v.shape) for k, v in self.T.items()})
        self.eng = q.Engine(self.spec, max_ctx=max_ctx, dtype=dtype, use_graph=use_graph).load_tensors(
            {k: words(v) for k, v in self.T.items()})
        self.batch = self.eng.batch(slots, max_ctx, page_tokens=page_tokens, n_pages=n_pages)
        self.vocab, self.dtype = vocab, dtype
        self.tol = REL32 if dtype == "float32" else REL16
        rel.rows = dtype != "float32"
        self.W64 = {k: np.asarray(v, dtype=np.float64) for k, v in self.T.items()}

    def tokens(self, n, low=0):
        return [int(t) for t in self.rng.integers(low, self.vocab, n)]

    def ref(self, toks, layers_out=None, W=None, cfg=None):
        return O.forward(cfg or self.cfg, W or self.W64, toks, layers_out)

    def close(self):
        self.batch.close()
        self.eng.close()


def rel(got, want):
    """Largest error of a logit over the logits' spread.  bf16 engines (REL16): root-mean-square errors of the rows
    instead - their 0.9-quantile, or a quarter of the worst row's, whichever is larger."""
    d = np.asarray(got, dtype=np.float64) - want
    if rel.rows:
        r = np.sqrt((d * d).mean(axis=-1)).reshape(-1) / (np.std(want) + 1e-30)
        return float(max(np.quantile(r, 0.9), r.max() / 4))
    return float(np.abs(d).max() / (np.std(want) + 1e-30))


rel.rows = False


def feed(m, slot, toks, cuts):
    """Feeds toks to `slot` in portions of the sizes in `cuts` (then one by one); logits of all rows."""
    out, pos = [], 0
    sizes = list(cuts)
    while pos < len(toks):
        n = min(sizes.pop(0) if sizes else 1, len(toks) - pos)
        out.append(m.batch.step([(slot, toks[pos:pos + n])], range(n)))
        pos += n
    return np.concatenate(out)


@pytest.fixture
def model():
    made = []

    def make(*a, **k):
        made.append(Model(*a, **k))
        return made[-1]
    yield make
    for m in made:
        m.close()


# ------------------------------------------------------------------ every mechanism alone, layer by layer
ALONE = {
    "ssm": [ssm()],
    "ssm-one-head": [ssm(heads=1, vdim=5, state=3, groups=1, conv=1, norm_groups=1)],
    "ssm-group-per-head-no-ff": [ssm(heads=3, vdim=8, state=16, groups=3, conv=2, norm_groups=1, mlp=None)],
    "ssm-wide-columns": [ssm(heads=2, vdim=70, state=33, groups=1, conv=5, norm_groups=4)],
    "ssm-large-state": [ssm(heads=2, vdim=9, state=130, groups=2, conv=4, norm_groups=2)],
    "ssm-huge-state": [ssm(heads=1, vdim=6, state=270, groups=1, conv=4, norm_groups=1)],
    "attention-only": [par(right=0.0)],
    "attention-mha-full-rotary": [par(heads=3, kv_heads=3, dim=10, vdim=22, rot_dims=10, right=0.0, keep=1)],
    "attention-one-key-head-no-rotary": [par(heads=5, kv_heads=1, dim=24, vdim=6, rot_dims=0, right=0.0, size=4, keep=6)],
    "attention-window-of-one": [par(right=0.0, size=1, keep=0)],
    "attention-window-of-one-keeps-one": [par(right=0.0, size=1, keep=1, mlp=None)],
    "attention-keeps-more-than-its-window": [par(right=0.0, size=3, keep=19)],
    "linear-only": [par(left=0.0)],
    "linear-one-head-tau-one": [par(left=0.0, rec_heads=1, rec_dim=4, rec_vdim=3, tau=1.0, rank=1)],
    "linear-wide": [par(left=0.0, rec_heads=2, rec_dim=40, rec_vdim=72, tau=16.0, rank=24, mlp=None)],
    "linear-large-key": [par(left=0.0, rec_heads=1, rec_dim=140, rec_vdim=20)],
    "linear-huge-key": [par(left=0.0, rec_heads=1, rec_dim=300, rec_vdim=10)],
    "both": [par()],
}


@pytest.mark.parametrize("name", sorted(ALONE))
@pytest.mark.parametrize("times", [0, 1, 3])
def test_each_mechanism_alone(model, name, times):
    m = model(ALONE[name], seed=3, loop=(0, 1, times) if times else None)
    toks = m.tokens(37)
    lay = []
    want = m.ref(toks, lay)
    m.batch.keep_layers(True)
    got = m.batch.step([(0, toks)], range(len(toks)))
    kept = m.batch.step_layers(len(toks))
    assert len(lay) == m.spec.n_runs == max(times, 1)
    for i, a in enumerate(lay):
        assert np.abs(kept[i] - a).max() < REL32 * max(np.abs(a).max(), 1.0), f"layer run {i}"
    assert rel(got, want) < m.tol
    m.batch.keep_layers(False)      # with the next run's norms fused
    assert rel(feed(m, 1, toks, [20, 2, 9]), want) < m.tol


@pytest.mark.parametrize("loop,width", [(None, 40), ((0, 5, 2), 40), ((1, 4, 2), 39), ((4, 5, 4), 44), ((0, 1, 3), 40), ((2, 2, 3), 40)])
def test_repeated_groups(model, loop, width):
    m = model(MIXED, seed=5, loop=loop, width=width)
    toks = m.tokens(45)
    lay = []
    want = m.ref(toks, lay)
    m.batch.keep_layers(True)
    got = m.batch.step([(0, toks)], range(len(toks)))
    kept = m.batch.step_layers(len(toks))
    for i, a in enumerate(lay):
        assert np.abs(kept[i] - a).max() < REL32 * np.abs(a).max(), f"layer run {i}"
    assert rel(got, want) < m.tol
    m.batch.keep_layers(False)
    assert rel(feed(m, 1, toks, [11, 2, 20]), want) < m.tol


@pytest.mark.parametrize("width", [40, 42])      # rows of whole 16-byte vectors, and rows that are not
def test_bf16_layers(model, width):
    m = model(MIXED, seed=5, dtype="bfloat16", loop=LOOP, width=width)
    toks = m.tokens(70)
    lay = []
    want = m.ref(toks, lay)
    m.batch.keep_layers(True)
    got = m.batch.step([(0, toks)], range(len(toks)))
    kept = m.batch.step_layers(len(toks))
    for i, a in enumerate(lay):
        assert np.sqrt(((kept[i] - a) ** 2).mean()) < REL16 * np.std(a), f"layer run {i}"
    assert rel(got, want) < m.tol


def test_scales_and_biases_reach_the_result(model):
    """Embedding scale, logit scale, biases, skip and mixer scales: the restatement itself tells each from its absence."""
    m = model([ssm(), par()], seed=11, embed_scale=5.5, logit_scale=0.37)
    toks = m.tokens(20)
    want = m.ref(toks)
    for key in ("l1.mix.left.q.b", "l1.mix.left.v.b", "l0.mix.conv.b", "l0.mix.D", "l1.mix.right.a2.b", "l0.mix.dt_bias"):
        assert rel(m.ref(toks, W=dict(m.W64, **{key: 0 * m.W64[key]})), want) > 20 * m.tol, key
    for change in (lambda c: c.update(logit_scale=1.0), lambda c: c["embedding"].update(scale=1.0),
                   lambda c: c["layers"][1]["mixer"].update(left_scale=1.0), lambda c: c["layers"][1]["mixer"].update(right_scale=1.0)):
        cfg = copy.deepcopy(m.cfg)
        change(cfg)
        assert rel(m.ref(toks, cfg=cfg), want) > 20 * m.tol
    assert rel(m.batch.step([(0, toks)], range(20)), want) < m.tol


def test_feed_forward_clamps(model):
    """Gate and up values far beyond the limit on both sides: the gate is cut above only, the up value on both sides."""
    def tweak(T, cfg):
        T["l0.mlp.gate"] *= np.float32(4.0)
        T["l0.mlp.up"] *= np.float32(4.0)
    m = model([ssm(mlp=dense(48, 0.75))], seed=2, tweak=tweak)
    toks = m.tokens(25)
    want = m.ref(toks)
    cfg = copy.deepcopy(m.cfg)
    cfg["layers"][0]["mlp"]["limit"] = 1e9
    assert rel(m.ref(toks, cfg=cfg), want) > 100 * m.tol
    assert rel(m.batch.step([(0, toks)], range(25)), want) < m.tol


# ------------------------------------------------------------------ schedules
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_prompt_equals_token_by_token_equals_portions(model, dtype):
    m = model(MIXED, seed=1, dtype=dtype, loop=LOOP)
    toks = m.tokens(75)
    want = m.ref(toks)
    whole = m.batch.step([(0, toks)], range(len(toks)))
    assert rel(whole, want) < m.tol
    one = feed(m, 1, toks, [])
    assert rel(one, want) < m.tol
    for slot, cuts in ((2, [2, 2, 3, 17, 2, 16, 1, 5, 20]), (3, [33, 2, 31, 2]), (0, [15, 1, 16, 2, 30])):
        m.batch.release(slot)
        assert rel(feed(m, slot, toks, cuts), want) < m.tol, cuts
    if dtype == "float32":      # the cut moves sums around, nothing else
        assert np.abs(one - whole).max() < 20 * REL32 * np.std(want)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_unequal_requests_in_one_step_equal_each_alone(model, dtype):
    m = model(MIXED, seed=4, dtype=dtype, loop=LOOP)
    seqs = [m.tokens(n) for n in (41, 3, 18, 29)]
    want = [m.ref(s) for s in seqs]
    got = [[] for _ in seqs]
    done = [0] * 4
    plan = [(7, 1, 2, 5), (1, 1, 16, 1), (17, 1, 0, 2), (2, 0, 0, 19), (14, 0, 0, 2)]
    for counts in plan:
        entries, spans = [], []
        for s, c in enumerate(counts):
            c = min(c, len(seqs[s]) - done[s])
            if c > 0:
                entries.append((s, seqs[s][done[s]:done[s] + c]))
                spans.append((s, c))
        rows = m.batch.step(entries, range(sum(c for _, c in spans)))
        at = 0
        for s, c in spans:
            got[s].append(rows[at:at + c])
            at += c
            done[s] += c
    for s in range(4):
        assert done[s] == len(seqs[s])
        assert rel(np.concatenate(got[s]), want[s]) < m.tol, f"request {s}"


def slow_decay(T, cfg):
    """Decays near one: what the first tokens wrote stays in the states."""
    for i, L in enumerate(cfg["layers"]):
        if L["type"] == "mamba2":
            T[f"l{i}.mix.A_log"][:] = -6.0
        else:
            T[f"l{i}.mix.right.a2.b"] += np.float32(6.0)


def fast_decay(T, cfg):
    """A mixture of channels (heads) that keep everything and channels that forget within a row or two."""
    for i, L in enumerate(cfg["layers"]):
        if L["type"] == "mamba2":
            T[f"l{i}.mix.A_log"][::2] = 3.5
            T[f"l{i}.mix.A_log"][1::2] = -5.0
        else:
            T[f"l{i}.mix.right.a2.b"][::3] = -60.0
            T[f"l{i}.mix.right.a2.b"][1::3] = 8.0


def test_pool_smaller_than_traffic_pages_slots_and_states_reused(model):
    layers = [ssm(heads=2, vdim=12, state=8, groups=1, conv=4, norm_groups=1), par(size=9, keep=2)]
    m = model(layers, seed=8, slots=2, page_tokens=16, n_pages=7, max_ctx=80, tweak=slow_decay, loop=(0, 2, 2))
    probe = m.tokens(40)
    other = [(probe[0] + 1) % m.vocab] + probe[1:]
    for k in (0, 1):              # each state alone carries token 0 to the last row (keep 0: the window does not)
        c = copy.deepcopy(m.cfg)
        c["layers"] = c["layers"][k:k + 1]
        c.pop("loop")
        if k == 1:
            c["layers"][0]["mixer"]["left"]["mask"]["keep_first"] = 0
        W1 = {n.replace(f"l{k}.", "l0."): v for n, v in m.W64.items() if n[0] != "l" or n.startswith(f"l{k}.")}
        a, b = O.forward(c, W1, probe), O.forward(c, W1, other)
        assert np.abs(a[-1] - b[-1]).max() > 1e-3 * np.std(a)
    for round_ in range(6):                                    # 6 pages for two slots: every page is used again
        seqs = [m.tokens(33 + round_), m.tokens(38 - round_)]
        want = [m.ref(s) for s in seqs]
        got = [feed(m, 0, seqs[0], [17, 2]), None]
        got[1] = feed(m, 1, seqs[1], [3, 30])
        for s in range(2):
            assert rel(got[s], want[s]) < m.tol, (round_, s)
            m.batch.release(s)
    with pytest.raises(Exception):
        m.batch.step([(0, m.tokens(70)), (1, m.tokens(70))], [0])     # more pages than the pool has: refused
    assert rel(feed(m, 0, probe, [40]), m.ref(probe)) < m.tol


BEACON = 1


def beacon(T, cfg):
    """One token whose key stands out for every query by a constant: q and k get a large bias along one unrotated
    coordinate, which only the beacon's embedding moves the key along; its value differs from the others'."""
    d = cfg["layers"][0]["mixer"]["left"]
    D = d["dim"]
    E = T["embed"]
    E[:, 0] = -0.5
    E[BEACON, 0] = 4.0
    T["l0.norm1"][0] = 1.0
    for h in range(d["kv_heads"]):
        T["l0.mix.left.k"][h * D + D - 1] = 0.0
        T["l0.mix.left.k"][h * D + D - 1, 0] = 1.0
        T["l0.mix.left.k.b"][h * D + D - 1] = 0.0
    for h in range(d["heads"]):
        T["l0.mix.left.q"][h * D + D - 1] = 0.0
        T["l0.mix.left.q.b"][h * D + D - 1] = 8.0
        T["l0.mix.left.q"][h * D:h * D + D - 1] *= np.float32(0.3)


@pytest.mark.parametrize("page_tokens,dim,vdim,dtype", [(16, 16, 12, "float32"), (64, 32, 32, "bfloat16"), (32, 64, 32, "bfloat16"),
                                                        (16, 32, 64, "bfloat16")])
@pytest.mark.parametrize("size,keep", [(5, 0), (16, 1), (30, 3), (32, 32), (33, 40), (64, 5), (70, 33)])
def test_window_edges_and_kept_first_tokens(model, page_tokens, dim, vdim, dtype, size, keep):
    """Beacons a little more than a window apart: the row where one is the window's last key and the next row tell the
    window's size; beacons as the last kept token and the first one behind tell keep_first - each asserted on the
    restatement, then in prompts, portions and decoding."""
    m = model([par(heads=4, kv_heads=1 if dim == 32 else 2, dim=dim, vdim=vdim, size=size, keep=keep, rot_dims=8, right=0.0, mlp=None)],
              seed=9, tweak=beacon, page_tokens=page_tokens, max_ctx=512, dtype=dtype, width=48)
    n = keep + 2 * size + 40
    base = m.tokens(n, low=2)
    toks = list(base)
    for p in range(keep + 3, n, size + 7):
        toks[p] = BEACON
    want = m.ref(toks)

    def with_mask(t, **kw):
        cfg = copy.deepcopy(m.cfg)
        cfg["layers"][0]["mixer"]["left"]["mask"].update(kw)
        return m.ref(t, cfg=cfg)
    shows = 20 * m.tol if dtype == "float32" else 3 * m.tol
    row_rel = lambda a, b: np.sqrt(((a - b) ** 2).mean(axis=-1)).max() / np.std(b)
    assert row_rel(with_mask(toks, size=size + 1), want) > shows
    if size > 1:
        assert row_rel(with_mask(toks, size=size - 1), want) > shows
    first = list(base)                          # beacons at the edge of the kept tokens
    first[keep] = BEACON
    kept = list(base)
    if keep:
        kept[keep - 1] = BEACON
        assert row_rel(with_mask(kept, keep_first=keep - 1)[keep + size:], m.ref(kept)[keep + size:]) > shows
    assert row_rel(with_mask(first, keep_first=keep + 1)[keep + size + 1:], m.ref(first)[keep + size + 1:]) > shows
    for t in (toks, first, kept):
        w = m.ref(t)
        for slot, cuts in ((0, [n]), (1, [keep + size - 1, 2, 2, 3]), (2, [n // 2, 2, 31])):
            m.batch.release(slot)
            got = feed(m, slot, t, cuts)
            assert row_rel(got, w) < m.tol, cuts


def test_far_first_tokens_through_many_pages(model):
    """Rows 300+ look 19 pages back at a kept first token, in prompts and decoding."""
    m = model([par(heads=4, kv_heads=2, size=24, keep=4, rot_dims=8, right=0.0, mlp=None)], seed=9, tweak=beacon, max_ctx=512, width=48)
    toks = m.tokens(330, low=2)
    toks[2] = BEACON
    want = m.ref(toks)
    moved = m.ref(toks[:2] + [5] + toks[3:])
    assert (np.abs(moved[300:] - want[300:]).max(axis=1) > 100 * m.tol * np.std(want)).all()
    assert rel(feed(m, 0, toks, [250, 13, 2, 2, 31, 2]), want) < m.tol
    assert rel(m.batch.step([(1, toks)], range(330)), want) < m.tol


def test_first_tokens_and_short_sequences(model):
    m = model(MIXED, seed=6, loop=LOOP)
    for n in (1, 2, 3, 4, 5):
        toks = m.tokens(n)
        assert rel(m.batch.step([(0, toks)], range(n)), m.ref(toks)) < m.tol
        m.batch.release(0)
        assert rel(feed(m, 0, toks, []), m.ref(toks)) < m.tol
        m.batch.release(0)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_long_decoding(model, dtype):
    m = model(MIXED, seed=7, dtype=dtype, tweak=slow_decay)
    toks = m.tokens(330)
    got = feed(m, 2, toks, [5])
    assert rel(got, m.ref(toks)) < m.tol


# ------------------------------------------------------------------ the recurrences' forms
REC = ["ssm", "ssm-one-head", "ssm-wide-columns", "ssm-large-state", "ssm-huge-state", "linear-only", "linear-one-head-tau-one",
       "linear-wide", "linear-large-key", "linear-huge-key"]


@pytest.mark.parametrize("name", REC)
@pytest.mark.parametrize("decay", [slow_decay, fast_decay])
def test_recurrences_in_tiles_and_pieces_equal_row_by_row(model, name, decay):
    """Portions of 9 rows and more run 16 rows at a time, portions above 128 in pieces with a carry; from fresh and kept
    states, ragged tiles and pieces, beside short entries.  Fast decays take the tiles whose decay leaves fp32's range."""
    m = model(ALONE[name], seed=21, max_ctx=512, tweak=decay)
    a, b = m.tokens(341), m.tokens(5)
    wa, wb = m.ref(a), m.ref(b)
    r1 = m.batch.step([(1, b[:3]), (0, a[:150])], range(153))
    r2 = m.batch.step([(0, a[150:]), (1, b[3:])], range(193))
    assert rel(np.concatenate([r1[3:], r2[:191]]), wa) < m.tol
    assert rel(np.concatenate([r1[:3], r2[191:]]), wb) < m.tol
    m.batch.release(0)
    assert rel(feed(m, 0, a, [129, 2, 17, 64, 9, 31, 33]), wa) < m.tol
    if decay is slow_decay:       # token 0 reaches the last row through the state alone
        moved = m.ref([(a[0] + 1) % m.vocab] + a[1:])
        assert np.abs(moved[-1] - wa[-1]).max() > 5 * m.tol * np.std(wa) or name == "ssm-one-head"


def test_long_prompts_beside_decoding(model):
    m = model([ssm(), par()], seed=12, max_ctx=1024, tweak=slow_decay, loop=(0, 2, 2))
    a, b = m.tokens(900), m.tokens(9)
    wa, wb = m.ref(a), m.ref(b)
    r1 = m.batch.step([(0, a[:600]), (1, b[:2])], range(602))
    r2 = m.batch.step([(1, b[2:]), (0, a[600:])], range(307))
    assert rel(np.concatenate([r1[:600], r2[7:]]), wa) < m.tol
    assert rel(np.concatenate([r1[600:], r2[:7]]), wb) < m.tol


def test_bf16_sizes_of_the_matrix_core_kernels(model):
    """Head sizes that are multiples of 32 and a width that is a multiple of 8: the shapes the bf16 engine's
    matrix-core products and attention kernels take."""
    layers = [ssm(heads=4, vdim=32, state=64, groups=2, conv=4, norm_groups=1, mlp=dense(96)),
              par(heads=4, kv_heads=1, dim=32, vdim=64, size=50, keep=7, rot_dims=16, rec_heads=2, rec_dim=32, rec_vdim=64, rank=8,
                  mlp=dense(96)),
              par(heads=6, kv_heads=2, dim=64, vdim=32, size=100, keep=40, rot_dims=64, rec_heads=2, rec_dim=64, rec_vdim=128, rank=16),
              par(heads=3, kv_heads=3, dim=128, vdim=128, size=40, keep=1, rot_dims=32, rec_heads=1, rec_dim=128, rec_vdim=32, rank=12)]
    m = model(layers, seed=13, dtype="bfloat16", width=64, page_tokens=64, max_ctx=640, loop=(1, 3, 2))
    toks = m.tokens(300)
    want = m.ref(toks)
    assert rel(m.batch.step([(0, toks)], range(300)), want) < m.tol
    assert rel(feed(m, 1, toks, [130, 2, 129, 17]), want) < m.tol


# ------------------------------------------------------------------ the serving entry points
def oracle_greedy(m, prompt, n):
    seq = list(prompt)
    for _ in range(n):
        seq.append(int(np.argmax(m.ref(seq)[-1])))
    return seq[len(prompt):]


def test_greedy_generation_through_the_batcher(model):
    """Five requests through ContinuousBatcher (two slots, a small page pool, 24-row steps): prompts are read in
    portions beside decoding requests; finished requests free their slot, pages and states for the waiting ones."""
    from qwen_inference_engine_amd.scheduler import ContinuousBatcher
    m = model(MIXED, seed=10, loop=LOOP)
    m.batch.close()
    cb = ContinuousBatcher(m.eng, slots=2, max_ctx=128, page_tokens=16, n_pages=9, chunk_tokens=24, keep_logits=True)
    m.batch = cb.batch
    prompts = [m.tokens(n) for n in (30, 5, 50, 1, 17)]
    gens = [6, 9, 4, 7, 5]
    rids = [cb.submit(p, g) for p, g in zip(prompts, gens)]
    out = cb.run()
    for p, g, rid in zip(prompts, gens, rids):
        want = oracle_greedy(m, p, g)
        got = out[rid]
        assert len(got) == g
        if got != want:   # a near-tie may flip: the logits must then be within rounding of the oracle's
            k = next(i for i in range(g) if got[i] != want[i])
            lg = m.ref(list(p) + want[:k])[-1]
            assert abs(lg[got[k]] - lg[want[k]]) < 1e-4 * np.std(lg), (rid, k)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_small_steps_replay_graphs_equal_eager(model, dtype):
    a = model(MIXED, seed=14, use_graph=True, dtype=dtype, loop=LOOP)
    b = model(MIXED, seed=14, use_graph=False, dtype=dtype, loop=LOOP)
    toks = a.tokens(60)
    for cuts in ([20, 3, 3, 3, 12, 12, 12], [9], [40, 1, 2]):      # replays with eager steps and releases in between
        ra, rb = feed(a, 0, toks, cuts), feed(b, 0, toks, cuts)
        assert np.array_equal(ra, rb)
        a.batch.release(0)
        b.batch.release(0)
    for _ in range(3):
        ra = a.batch.step([(0, toks[:2]), (1, toks[2:3])], range(3))
        rb = b.batch.step([(0, toks[:2]), (1, toks[2:3])], range(3))
        assert np.array_equal(ra, rb)
    assert a.batch.graph_stats()[0] >= 1 and a.batch.graph_stats()[1] >= 30 and b.batch.graph_stats()[0] == 0


def save_model(m, path):
    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump({k: v for k, v in m.cfg.items() if not k.startswith("_")}, f)
    hdr, blobs, off = {}, [], 0
    for k, v in m.T.items():
        b = words(v).tobytes()
        hdr[k] = {"dtype": "BF16", "shape": list(v.shape), "data_offsets": [off, off + len(b)]}
        blobs.append(b)
        off += len(b)
    h = json.dumps(hdr).encode()
    with open(os.path.join(path, "model.safetensors"), "wb") as f:
        f.write(len(h).to_bytes(8, "little") + h + b"".join(blobs))


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_trace_replay_and_generation_command_lines(model, tmp_path, dtype):
    m = model(MIXED if dtype == "float32" else MIXED[:3], seed=15, dtype=dtype, loop=LOOP if dtype == "float32" else None)
    save_model(m, str(tmp_path / "model"))
    a, b = m.tokens(50), m.tokens(21)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:30], "want": [0, 29]}, {"id": "b", "tokens": b[:2], "want": []}], "end": []},
             {"step": 1, "entries": [{"id": "b", "tokens": b[2:], "want": [18]}, {"id": "a", "tokens": a[30:31], "want": [0]}], "end": ["b"]},
             {"step": 2, "entries": [{"id": "a", "tokens": a[31:], "want": [18]}], "end": ["a"]}]
    out = tmp_path / "out"
    r = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model", str(tmp_path / "model"), "--dtype", dtype,
                        "--out", str(out), "--max-tokens", "192"], input="\n".join(json.dumps(s) for s in steps) + "\n",
                       capture_output=True, text=True, timeout=300)
    assert r.returncode == 0, r.stderr[-2000:]
    assert [ln for ln in r.stdout.split("\n") if ln.startswith("done")] == ["done 0", "done 1", "done 2"]
    wa, wb = m.ref(a), m.ref(b)
    got = [np.fromfile(out / f"{i}.f32", dtype="<f4").reshape(-1, m.vocab) for i in range(3)]
    assert rel(got[0], wa[[0, 29]]) < m.tol
    assert rel(got[1], np.stack([wb[20], wa[30]])) < m.tol
    assert rel(got[2], wa[[49]]) < m.tol
    if dtype == "float32":
        r = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "qie"), "--model", str(tmp_path / "model"), "--dtype", "float32",
                            "--gen", "5", "--prompt", ",".join(map(str, b)), "--prompt", " ".join(map(str, a[:7])), "--slots", "2",
                            "--chunk-tokens", "16"], capture_output=True, text=True, timeout=300)
        assert r.returncode == 0, r.stderr[-2000:]
        got = {ln.split(":")[0]: [int(t) for t in ln.split(":")[1].split()] for ln in r.stdout.splitlines() if ln.startswith("tokens[")}
        assert got["tokens[0]"] == oracle_greedy(m, b, 5)
        assert got["tokens[1]"] == oracle_greedy(m, a[:7], 5)


# ------------------------------------------------------------------ the new pieces beside other designs' pieces
@pytest.mark.parametrize("block", ["parallel", "prenorm"])
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_blocks_and_mixers_combine(block, dtype):
    """The parallel block around every mixer and a routed feed-forward, the state space inside the pre-norm block: a
    model no reader makes, restated with the designs' oracles; portions above and below the branch threshold."""
    import lugipel_oracle as LO
    import nodutar_oracle as NO
    import qwen_inference_engine_amd as q
    import verelorn_oracle as VO
    from qwen_inference_engine_amd import spec as S
    W, V, eps, n = 48, 83, 1e-5, 150
    ff = lambda act, **k: S.FeedForward("dense", 32, act=act, **k)
    layers = [S.LayerSpec(S.StateSpace(4, 8, 12, 2, 3, 2), ff("clamped_gated", limit=1.0)),
              S.LayerSpec(S.MinGru(40), ff("gelu_tanh_gated")),
              S.LayerSpec(S.ChannelDelta(2, 1, 8, 16, 3, 4, 4), ff("silu_gated")),
              S.LayerSpec(S.LatentAttention(2, 8, 4, 8, 16, 0, 4, 100.0, 0.3, None, 8, "interleaved", False), ff("clamped_gated", limit=0.5)),
              S.LayerSpec(S.StateSpace(2, 24, 16, 1, 4, 1), S.FeedForward("moe", 16, 4, 2, "softmax_out"))]
    if block == "parallel":
        layers.append(S.LayerSpec(S.AttentionWithRecurrence(
            S.GqaAttention(4, 2, 8, 8, 0.3, qk_norm="weight", rot_dims=4, rot_base=100.0, rot_layout="interleaved", rot_values=True,
                           mask="chunk", mask_size=9), S.GatedRecurrence(2, 8, 8), 0.8, 1.1), None))
    spec = S.LayeredSpec("mix", W, V, eps, tuple(layers), False, block=block, tied_head=True, embed_scale=2.0, logit_scale=0.5)
    rng = np.random.default_rng(3)
    T = {}
    for name, shape in spec.tensor_shapes().items():
        if name.endswith(("norm", "norm1", "norm2", ".D")):
            v = 1.0 + 0.2 * rng.standard_normal(shape)
        elif name.endswith("lower"):
            v = rng.uniform(0.1, 0.9, shape)
        elif len(shape) == 1:
            v = 0.3 * rng.standard_normal(shape)
        else:
            v = rng.standard_normal(shape) * (0.4 if name.endswith((".o", "down")) else 0.5 if name == "embed" else 1.0) / \
                (np.sqrt(shape[-1]) if name != "embed" else 1.0)
        T[name] = O.to_bf16_exact(v)
    D = {k: v.astype(np.float64) for k, v in T.items()}

    def mixer(i, h):
        m, p = layers[i].mixer, f"l{i}.mix."
        if isinstance(m, S.StateSpace):
            return O.state_space({k: getattr(m, k) for k in ("heads", "vdim", "state", "groups", "norm_groups")}, D, p, h, eps)
        if isinstance(m, S.MinGru):
            return LO.min_gru(h, D, p)[0]
        if isinstance(m, S.ChannelDelta):
            return VO.channel_delta({k: getattr(m, k) for k in ("heads", "kv_heads", "dim", "vdim")}, D, p, h, eps)
        if isinstance(m, S.LatentAttention):
            c = {"heads": m.heads, "dim": m.dim, "rot_dim": m.rot_dim, "vdim": m.vdim, "kv_rank": m.kv_rank, "scale": m.scale,
                 "rot": {"base": 100.0, "dims": 4}}
            return VO.latent_attention(c, D, p, h, eps, VO.latent_kv(c, D, p, h, eps))
        a, c = m.attn, m.rec
        cfg = {"left_scale": 0.8, "right_scale": 1.1, "right": {"heads": c.heads, "dim": c.dim, "vdim": c.vdim},
               "left": {"heads": a.heads, "kv_heads": a.kv_heads, "dim": a.dim, "vdim": a.vdim, "scale": a.scale,
                        "mask": {"size": 9}, "rot": {"base": 100.0, "dims": 4}}}
        return NO.parallel_mixer(h, cfg, D, p, eps)

    def feed_forward(i, h):
        f, p = layers[i].mlp, f"l{i}.mlp."
        if f.kind == "moe":
            return NO.moe_ff(h, {"router": {"experts": 4, "top": 2}}, D, p)
        if f.act == "clamped_gated":
            return O.clamped_ff({"limit": f.limit}, D, p, h)
        if f.act == "gelu_tanh_gated":
            return VO.dense_ff(D, p, h)
        return (O.silu(h @ D[p + "gate"].T) * (h @ D[p + "up"].T)) @ D[p + "down"].T

    toks = [int(t) for t in rng.integers(0, V, n)]
    x = D["embed"][toks] * 2.0
    for i, L in enumerate(layers):
        y = mixer(i, O.norm(x, D[f"l{i}.norm1"], eps))
        z = x if block == "parallel" else x + y
        f = feed_forward(i, O.norm(z, D[f"l{i}.norm2"], eps)) if L.mlp is not None else 0.0
        x = x + y + f
    want = O.norm(x, D["final.norm"], eps) @ D["embed"].T * 0.5
    eng = q.Engine(spec, max_ctx=256, dtype=dtype).load_tensors({k: words(v) for k, v in T.items()})
    b = eng.batch(2, 256, page_tokens=32)
    rel.rows = dtype != "float32"
    for slot, cuts in ((0, [n]), (1, [70, 2, 66, 3])):
        got, pos = [], 0
        while pos < n:
            c = min(cuts.pop(0) if cuts else 1, n - pos)
            got.append(b.step([(slot, toks[pos:pos + c])], range(c)))
            pos += c
        assert rel(np.concatenate(got), want) < (REL32 if dtype == "float32" else REL16)
    b.close()
    eng.close()
