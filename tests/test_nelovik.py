"""Nelovik against a plain implementation of its equations
(tests/helpers/nelovik_plain.py): each mechanism alone, then whole models
through the engine -- prompts cut in every way, mixed batches, reused pages
and slots, greedy generation. Each case runs on the CPU reference operations
and, marked gpu, on the kernels in 32-bit and bf16."""

import io
import json
import os
import subprocess
import sys

import pytest
import torch

sys.path.insert(0, os.path.join(os.path.dirname(__file__), "helpers"))

import nelovik_cases as cases  # noqa: E402
import nelovik_plain as plain  # noqa: E402
from lm_cases import (check_trace, engine, error,  # noqa: E402
                      feed_in_portions, generate, greedy,
                      mixed_batches_error, name_of, open_sequence, padded,
                      portions_of, rel, tokens_for, trace_lines, write_model)

from clearml_serving_amd.engines.llm.token_batch import TokenBatch  # noqa: E402
from clearml_serving_amd.models.mixers import (DenseMlp,  # noqa: E402
                                               GatedDelta, GroupedAttention,
                                               GroupedAttentionMixer,
                                               ParallelMixer, RecurrentMixer,
                                               StateSpace)
from clearml_serving_amd.ops import grouped, linear_state, lm  # noqa: E402

REPO = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))

CPU = pytest.param("cpu", torch.float32, 2e-5, id="cpu")
GPU32 = pytest.param("cuda:0", torch.float32, 2e-5, id="gpu-fp32",
                     marks=pytest.mark.gpu)
GPU16 = pytest.param("cuda:0", torch.bfloat16, 4e-2, id="gpu-bf16",
                     marks=pytest.mark.gpu)
ALL = pytest.mark.parametrize("device,dtype,tol", [CPU, GPU32, GPU16])
# whole models: rounding grows from layer to layer
MODEL = pytest.mark.parametrize("device,dtype,tol", [
    pytest.param("cpu", torch.float32, 1e-4, id="cpu"),
    pytest.param("cuda:0", torch.float32, 1e-4, id="gpu-fp32",
                 marks=pytest.mark.gpu),
    pytest.param("cuda:0", torch.bfloat16, 8e-2, id="gpu-bf16",
                 marks=pytest.mark.gpu)])
EPS = 1e-5


def double(st):
    return {k: v.double() for k, v in st.items()}


def random_state(shapes, seed, sharp=2.5):
    g = torch.Generator().manual_seed(seed)
    return {k: cases.random_tensor(k, s, g, sharp).to(torch.bfloat16)
            for k, s in shapes.items()}


def inputs(n, width, seed):
    g = torch.Generator().manual_seed(seed)
    return torch.randn(n, width, generator=g).to(torch.bfloat16)


# --------------------------------------------------------------------- #
# around the sublayers
# --------------------------------------------------------------------- #
@ALL
@pytest.mark.parametrize("width", [44, 300, 2080, 5000])
@pytest.mark.parametrize("branches", [0, 1, 2])
@pytest.mark.parametrize("norms", [0, 1, 2])
def test_sublayers_into_the_stream(device, dtype, tol, width, branches,
                                   norms):
    n, eps, wp = 5, 1e-2, lm.pad32(width)
    g = torch.Generator().manual_seed(width + branches)
    x = torch.randn(n, width, generator=g)
    x[2] *= 1e-2  # eps matters here
    made = [torch.randn(n, width, generator=g).to(dtype) for _ in range(3)]
    made[1][3] *= 1e-2
    w = [torch.randn(width, generator=g).to(dtype) for _ in range(4)]
    want = x.double() + sum(
        0.5 * plain.over_rms(o.double(), eps) * v.double()
        for o, v in zip(made[1:1 + branches], w))
    plain_too = branches != 1
    if plain_too:
        want = want + made[0].double()
    xs = padded(x, wp).to(device)

    def put(v):
        return padded(v, wp).to(device)

    h = lm.add_branches(
        xs, put(made[0]) if plain_too else None,
        [(put(o), put(v)) for o, v in zip(made[1:1 + branches], w)], 0.5,
        [lm.RowNorm(put(v), width, eps, 0.0) for v in w[2:2 + norms]], width,
        eps, dtype)
    # the stream is 32-bit whatever the product type is
    assert xs.dtype == torch.float32 and len(h) == norms
    assert rel(xs[:, :width], want) < 1e-5
    for got, v in zip(h, w[2:]):
        assert got.dtype == dtype
        assert rel(got[:, :width], plain.over_rms(want, eps)
                   * v.double()) < max(tol, 1e-5)
        if wp > width:
            assert got[:, width:].abs().max() == 0
    if wp > width:
        assert xs[:, width:].abs().max() == 0


@ALL
@pytest.mark.parametrize("norms", [1, 2])
def test_embedding(device, dtype, tol, norms):
    vocab, width, wp, eps = 9, 40, 64, 1e-3
    g = torch.Generator().manual_seed(3)
    table = torch.randn(vocab, width, generator=g).to(dtype)
    w = [torch.randn(width, generator=g).to(dtype) for _ in range(norms)]
    toks = torch.tensor([3, 0, 8, 3])
    x, h = lm.embed_norms(
        toks.to(device), padded(table, wp).to(device),
        [lm.RowNorm(padded(v, wp).to(device), width, eps, 0.0) for v in w])
    x0 = table.double()[toks]
    assert x.dtype == torch.float32 and len(h) == norms
    assert rel(x[:, :width], x0) == 0
    for got, v in zip(h, w):
        assert rel(got[:, :width], plain.over_rms(x0, eps) * v.double()) \
            < max(tol, 1e-5)


@ALL
@pytest.mark.parametrize("p,q", [(0.8, 0.8), (-3.0, 4.0), (2.0, -20.0)])
def test_activation(device, dtype, tol, p, q):
    z = torch.linspace(-30, 6, 32 * 40).view(40, 32)
    z[0, :6] = torch.tensor([0.0, 1e-4, -1e-4, -0.5, -0.499, -1e-2])
    z = z.to(dtype)
    mod = DenseMlp(8, 32)
    mod.act.data = torch.tensor([p, q])
    mod.finalize()
    out = torch.full((40, 96), 7.0, dtype=dtype, device=device)
    lm.xielu(z.to(device), mod._coef.to(device), out[:, 32:64])
    want = plain.xielu(z.double(), torch.tensor(p).double(),
                       torch.tensor(q).double())
    got = out[:, 32:64].double().cpu()
    # one by one: what is small is right too (it is zero somewhere below 0)
    err = (got - want).abs() / (want.abs() + 0.3 * z.double().abs() + 1e-9)
    assert err.max() < (1e-5 if dtype == torch.float32 else 1e-2)
    assert (out[:, :32] == 7).all() and (out[:, 64:] == 7).all()


@ALL
@pytest.mark.parametrize("width,ff", [(44, 30), (64, 96), (33, 1)])
def test_feed_forward(device, dtype, tol, width, ff):
    st = random_state({"up": (ff, width), "down": (width, ff), "act": (2,)},
                      ff)
    mod = DenseMlp(width, ff)
    assert mod.shapes() == {k: tuple(v.shape) for k, v in st.items()}
    mod.pack(st.__getitem__)
    down = torch.zeros(lm.pad32(width), mod.out_cols)
    mod.pack_out(down, st.__getitem__)
    mod = mod.to(device).to(dtype)
    mod.finalize()
    h = inputs(50, width, 1)
    out = torch.empty(50, mod.out_cols, dtype=dtype, device=device)
    mod.context(padded(h, lm.pad32(width)).to(dtype).to(device), out)
    got = out.float().cpu() @ down.T
    assert rel(got[:, :width], plain.dense(h.double(), double(st))) < tol


# --------------------------------------------------------------------- #
# running one mixer on a sequence
# --------------------------------------------------------------------- #
def caches_for(mod, n_pages, block_size, slots, device, dtype):
    """filled with what earlier owners may have left"""
    def make(kind, *dims):
        if kind == "both":
            return tuple(make(*d) for d in dims)
        if kind == "paged":
            rows = grouped.page_rows(block_size, *dims[1:] or (0,))
            return torch.full((n_pages, rows, dims[0]), 3.0, dtype=dtype,
                              device=device)
        return tuple(torch.full((slots, *s), 2.0, device=device, dtype=t)
                     for s, t in zip(dims, (torch.float32, dtype)))
    return make(*mod.cache_layout())


def run_mixer(mod, h, portions, device, dtype, block_size=4, absorb_max=None,
              pages=None, forward=None):
    """one sequence through a mixer in portions -> [n, width] float64"""
    mod = mod.to(device).to(dtype)
    mod.finalize()
    n = h.shape[0]
    pages = pages or list(range(-(-n // block_size)))
    cache = caches_for(mod, max(pages) + 1, block_size, 3, device, dtype)
    views = sorted({m.view for m in mod.modules()
                    if isinstance(m, GroupedAttention)}, key=str)
    out, at = [], 0
    for k in portions:
        _, batch, _ = TokenBatch.build(
            {"tokens": [[0] * k], "starts": [at], "blocks": [pages],
             "state_slots": [1], "want": [[]]}, block_size, device,
            tile=64, absorb_max=absorb_max, windows=views)
        x = padded(h[at:at + k], lm.pad32(h.shape[1])).to(dtype).to(device)
        y = mod(x, batch, cache, {}) if forward is None else \
            forward(mod, x, batch, cache)
        out.append(y.double().cpu())
        at += k
    assert at == n
    return torch.cat(out)[:, :h.shape[1]]


# absorbed: every token reads the cache rows; expanded: tiles of queries
FORMS = pytest.mark.parametrize("absorb_max", [None, 1],
                                ids=["absorbed", "expanded"])


def skip_expanded_in_32_bit(absorb_max, device, dtype):
    if absorb_max is not None and device != "cpu" and dtype == torch.float32:
        pytest.skip("every token reads the cache rows in 32-bit")


# --------------------------------------------------------------------- #
# windowed attention over pooled history
# --------------------------------------------------------------------- #
def attention_args(m, width, eps):
    r = m["rot"]
    return (width, m["heads"], m["kv_heads"], m["dim"], m["vdim"],
            m["scale"], eps), dict(
        rot=(r["base"], r["dims"], 1.0), rot_half=True,
        window=m["mask"]["size"], pool=m["mask"]["pool"], cap=m["softcap"],
        qk_norm="all", sink="learned", bias=True)


def attention_of(m, width, st, eps=EPS):
    args, kw = attention_args(m, width, eps)
    mod = GroupedAttentionMixer(*args, **kw)
    assert mod.shapes() == cases.attention_shapes(m, width)
    mod.pack(st.__getitem__)
    return mod


WINDOWS = [
    dict(), dict(heads=1, kv=1, dim=2, vdim=1, rot=2, size=1, pool=1),
    dict(heads=20, kv=1, dim=40, vdim=33, rot=34, size=64, pool=7),
    dict(heads=4, kv=4, dim=128, vdim=64, rot=32, size=65, pool=32, cap=25.0),
    dict(heads=6, kv=3, dim=64, vdim=128, rot=64, size=100, pool=1, cap=2.0),
    dict(heads=2, kv=2, dim=200, vdim=250, rot=8, size=33, pool=50),
    dict(heads=8, kv=2, dim=64, vdim=64, rot=32, size=16, pool=2,
         base=1e4),
]


@ALL
@FORMS
@pytest.mark.parametrize("size", range(len(WINDOWS)))
def test_window_attention(device, dtype, tol, absorb_max, size):
    skip_expanded_in_32_bit(absorb_max, device, dtype)
    m = cases.left(**WINDOWS[size])
    m["scale"] = m["dim"] ** -0.5
    n, width = 300, 36
    st = random_state(cases.attention_shapes(m, width), size, 1.5)
    h = inputs(n, width, size)
    h[1] *= 1e-2  # eps of the norms matters here
    want = plain.window_attention(h.double(), double(st), m, EPS)
    mod = attention_of(m, width, st)
    pages = [4 * (i % 5) + i // 5 for i in range(20)]  # in no order
    for portions in ([n], portions_of(n, [131, 2, 1, 40])):
        got = run_mixer(mod, h, portions, device, dtype, 16, absorb_max,
                        pages)
        assert rel(got, want) < tol
    # the oracle with one thing wrong is told apart
    wrong = dict(double(st), sink=st["sink"].double() - 3.0)
    assert rel(plain.window_attention(h.double(), wrong, m, EPS),
               want) > 1e-2
    wrong = dict(double(st), **{"v.b": 0 * st["v.b"].double()})
    assert rel(plain.window_attention(h.double(), wrong, m, EPS),
               want) > 1e-2


def needle(st, h, m, key, query):
    """the query at `query` scores the key at `key` far above all others, by
    the first channel that is not rotated; values tell the keys apart"""
    d = m["rot"]["dims"]
    h[:, :2] = 0
    h[key, 0] = h[query, 1] = 12.0
    for k in ("q", "k"):
        st[k] *= 0.05
        st[k + ".b"] *= 0.05
        st[k][:, :2] = 0
        st[k + ".norm"].fill_(1.0)
    st["v"][:, :2] = 0
    for a in range(m["heads"]):
        st["q"][a * m["dim"] + d] = 0
        st["q"][a * m["dim"] + d, 1] = 1.0
    for a in range(m["kv_heads"]):
        st["k"][a * m["dim"] + d] = st["k.b"][a * m["dim"] + d] = 0
        st["k"][a * m["dim"] + d, 0] = 1.0
    st["sink"].abs_()


@ALL
@FORMS
@pytest.mark.parametrize("size,pool,block_size", [
    (11, 4, 4), (70, 3, 4), (64, 16, 16), (5, 24, 16), (40, 1, 8)])
def test_edges_of_windows_and_blocks(device, dtype, tol, absorb_max, size,
                                     pool, block_size):
    """a key that stands out: just inside and outside of the window, in the
    last block that is seen and the first that is not yet, and far away; the
    query in a prompt, decoded, and at the start of a portion"""
    skip_expanded_in_32_bit(absorb_max, device, dtype)
    m = cases.left(heads=4, kv=2, dim=20, vdim=12, rot=6, size=size,
                   pool=pool, cap=60.0, scale=0.8 + 0.4 * pool)
    n, width = 140, 36
    for query in (n - 1, n - 30):
        lo = query - size + 1
        seen = lo // pool  # blocks
        keys = {lo: -1, lo - 1: 1, 0: 0, pool: 0}  # key: other window
        if seen:
            keys[seen * pool - 1] = keys[(seen - 1) * pool] = 0
        if seen * pool < lo:  # left the window, its block is not seen yet
            keys[seen * pool] = None
        for key, change in keys.items():
            st = random_state(cases.attention_shapes(m, width), 4)
            h = inputs(n, width, key)
            needle(st, h, m, key, query)
            want = plain.window_attention(h.double(), double(st), m, EPS)
            mod = attention_of(m, width, st)
            cuts = ([n], [query - 3] + [1] * (n - query + 3),
                    [query] + [n - query], portions_of(n, [67, 2]))
            for portions in cuts[:2] if device == "cpu" else cuts:
                got = run_mixer(mod, h, portions, device, dtype, block_size,
                                absorb_max)
                assert rel(got[query], want[query]) < tol
                if dtype == torch.float32:  # such scores amplify rounding
                    assert rel(got, want) < tol
            if change is None:  # the key does not count at all
                h2 = h.clone()
                h2[key, 0] = 0
                off = plain.window_attention(h2.double(), double(st), m, EPS)
                assert rel(off[query], want[query]) < 1e-9
            elif change:
                if pool == 1:  # a block of one is its token
                    continue
                off = plain.window_attention(
                    h.double(), double(st),
                    dict(m, mask={"size": size + change, "pool": pool}), EPS)
                assert rel(off[query], want[query]) > 1e-2
            elif device == "cpu":  # without the blocks it would be lost
                off = plain.window_attention(
                    h.double(), double(st),
                    dict(m, mask={"size": size, "pool": 1000}), EPS)
                assert rel(off[query], want[query]) > 1e-2


def test_pages_with_pooled_rows():
    for bs in (1, 4, 16, 17):
        for pool in (0, 1, 2, 3, 5, 16, 31):
            rows = grouped.page_rows(bs, pool)
            assert grouped.page_tokens(rows, pool) == bs
            # every block's row is its own, in the page of its last token
            used = set()
            for p in range(pool - 1, 20 * bs, pool) if pool else ():
                r = grouped.pooled_row(p // bs, p % bs, bs, pool)
                assert r // rows == p // bs and r % rows >= bs
                assert r not in used
                used.add(r)
            for p in range(3 * bs):
                r = grouped.token_row(p // bs, p % bs, bs, pool)
                assert r // rows == p // bs and r not in used


def test_halves_are_brought_together():
    """scores do not depend on the channels' order, rotated ones included"""
    m = cases.left(dim=12, rot=6)
    st = random_state(cases.attention_shapes(m, 36), 1)
    order = attention_of(m, 36, st).attn.order.tolist()
    assert order == [0, 3, 1, 4, 2, 5, 6, 7, 8, 9, 10, 11]


@pytest.mark.parametrize("kw,what", [
    (dict(pool=4), "window"), (dict(window=8, pool=4, keep=2), "pooled"),
    (dict(window=8, pool=4, values_are_keys=True), "values"),
    (dict(qk_norm="all", values_are_keys=True), "values")])
def test_combinations_without_a_kernel_are_refused(kw, what):
    with pytest.raises(ValueError, match=what):
        GroupedAttention(32, 4, 2, 8, 8, 1.0, **kw)


# --------------------------------------------------------------------- #
# recurrences
# --------------------------------------------------------------------- #
def delta_of(m, width, st, eps=EPS):
    mod = RecurrentMixer(width, GatedDelta(
        width, m["heads"], m["kv_heads"], m["dim"], m["vdim"], m["conv"],
        eps))
    assert mod.shapes() == cases.delta_shapes(m, width)
    return packed(mod, st)


def space_of(m, width, st, eps=EPS):
    mod = RecurrentMixer(width, StateSpace(
        width, m["heads"], m["vdim"], m["state"], m["groups"], m["conv"],
        m["norm_groups"], eps))
    assert mod.shapes() == cases.state_shapes(m, width)
    return packed(mod, st)


def packed(mod, st):
    mod.pack(st.__getitem__)
    mod.o = torch.nn.Parameter(
        torch.zeros(mod.inp.shape[1], mod.out_cols), requires_grad=False)
    mod.pack_out(mod.o.data, st.__getitem__)
    return mod


def with_output(mod, x, batch, cache):
    ctx = x.new_empty(x.shape[0], mod.out_cols)
    mod.context(x, batch, cache, ctx)
    return ctx @ mod.o.T


DELTAS = [
    dict(), dict(heads=1, kv=1, dim=1, vdim=1, conv=1),
    dict(heads=3, kv=3, dim=64, vdim=64, conv=2),
    dict(heads=2, kv=1, dim=33, vdim=70, conv=3),
    dict(heads=4, kv=2, dim=96, vdim=40, conv=8),
    dict(heads=2, kv=2, dim=128, vdim=128, conv=4),
    dict(heads=2, kv=1, dim=150, vdim=200, conv=5),
    dict(heads=33, kv=11, dim=8, vdim=12, conv=4),
]
CUTS = ([200], [1] * 200, [17, 2, 1, 16, 3, 32, 33, 31, 65],
        [64, 2, 30, 2, 2, 100])


@ALL
@pytest.mark.parametrize("size", range(len(DELTAS)))
def test_delta_rule(device, dtype, tol, size):
    m, n, width = cases.delta(**DELTAS[size]), 200, 36
    st = random_state(cases.delta_shapes(m, width), size)
    h = inputs(n, width, size)
    h[5] *= 1e-2  # eps of the unit vectors and of the norm matters here
    eps = 1e-2 if m["vdim"] < 3 else EPS
    want = plain.delta_rule(h.double(), double(st), m, eps)
    mod = delta_of(m, width, st, eps)
    for portions in CUTS:
        got = run_mixer(mod, h, portions_of(n, portions), device, dtype,
                        forward=with_output)
        assert rel(got, want) < tol, portions[:3]


SPACES = [
    dict(), dict(heads=1, vdim=1, state=1, groups=1, conv=1, parts=1),
    dict(heads=8, vdim=64, state=128, groups=8, conv=4, parts=8),
    dict(heads=5, vdim=33, state=70, groups=1, conv=8, parts=11),
    dict(heads=2, vdim=128, state=64, groups=2, conv=2, parts=1),
    dict(heads=4, vdim=200, state=30, groups=2, conv=5, parts=32),
    dict(heads=33, vdim=8, state=16, groups=3, conv=4, parts=1),
    dict(heads=2, vdim=24, state=256, groups=1, conv=3, parts=16),
]


@ALL
@pytest.mark.parametrize("size", range(len(SPACES)))
def test_state_space(device, dtype, tol, size):
    m, n, width = cases.right(**SPACES[size]), 200, 36
    st = random_state(cases.state_shapes(m, width), size)
    h = inputs(n, width, size)
    h[5] *= 1e-2
    eps = 1e-2 if m["heads"] * m["vdim"] < 3 * m["norm_groups"] else EPS
    want = plain.state_space(h.double(), double(st), m, eps)
    mod = space_of(m, width, st, eps)
    for portions in CUTS:
        got = run_mixer(mod, h, portions_of(n, portions), device, dtype,
                        forward=with_output)
        assert rel(got, want) < tol, portions[:3]


@pytest.mark.parametrize("device,dtype,tol", [GPU32, GPU16])
@pytest.mark.parametrize("kind,size,seg", [
    ("delta", 0, 1), ("delta", 2, 2), ("delta", 4, 1), ("delta", 5, 3),
    ("delta", 6, 1), ("space", 0, 1), ("space", 2, 2), ("space", 5, 3),
    ("space", 7, 1)])
def test_recurrences_in_segments(device, dtype, tol, kind, size, seg,
                                 monkeypatch):
    """long portions are cut, and walked from the states in front of the
    segments; portions end inside, at and right behind a segment's end"""
    monkeypatch.setattr(linear_state, "segment_tiles", lambda *a: seg)
    n, width = 600, 36
    if kind == "delta":
        m, make, ref = cases.delta(**DELTAS[size]), delta_of, plain.delta_rule
        st = random_state(cases.delta_shapes(m, width), size)
    else:
        m, make, ref = cases.right(**SPACES[size]), space_of, \
            plain.state_space
        st = random_state(cases.state_shapes(m, width), size)
    st["A_log"] -= 2.0  # what the first segment leaves lasts
    h = inputs(n, width, size)
    want = ref(h.double(), double(st), m, EPS)
    mod = make(m, width, st)
    for portions in ([n], [128, 2, 192, 65, 1, 212], [5, 64, 531]):
        assert rel(run_mixer(mod, h, portions, device, dtype,
                             forward=with_output), want) < tol


def test_which_portions_are_cut():
    def cut(tiles, seqs, heads, vdim):
        return linear_state.segment_tiles(tiles, seqs, linear_state.StateSpec(
            True, heads, heads, 64, vdim, 4, heads, EPS))

    assert cut(0, 0, 4, 64) == 0  # none
    assert cut(4, 1, 4, 64) == 0  # short
    assert cut(4000, 16, 16, 64) == 0  # enough of them
    for tiles, seqs, heads, vdim in ((128, 1, 16, 128), (128, 4, 16, 64),
                                     (2000, 1, 1, 256)):
        assert 2 <= cut(tiles, seqs, heads, vdim) < tiles / seqs


@pytest.mark.parametrize("device,dtype,tol", [CPU, GPU32])
@pytest.mark.parametrize("kind", ["forgets", "keeps", "same keys"])
def test_delta_rule_extremes(device, dtype, tol, kind):
    """decays that end the state at every token or never, and keys that are
    all alike, written at full rate"""
    m, n, width = cases.delta(2, 1, 24, 20, 3), 150, 36
    st = random_state(cases.delta_shapes(m, width), 3)
    h = inputs(n, width, 9)
    if kind == "forgets":
        st["A_log"].fill_(4.0)
        st["dt_bias"].fill_(5.0)
    else:
        st["A_log"].fill_(-9.0)
    if kind == "same keys":
        h[:, 0] = 8.0
        st["k"][:, 1:] = 0
        st["b"].zero_()
        st["b"][:, 0] = 4.0
    want = plain.delta_rule(h.double(), double(st), m, EPS)
    mod = delta_of(m, width, st)
    for portions in ([n], [1] * n, portions_of(n, [33, 2])):
        got = run_mixer(mod, h, portions, device, dtype, forward=with_output)
        assert rel(got, want) < 10 * tol


def test_recurrence_oracles_tell_faults_apart():
    """decay, then removal and write, then read-out: another order shows, and
    so does a lost state or convolution input"""
    g = torch.Generator().manual_seed(0)
    q, k, v = (torch.randn(40, 8, generator=g).double() for _ in range(3))
    k = plain.unit(k)
    w, b = torch.rand(2, 40, generator=g).double()
    want, _ = plain.delta_scan(q, k, v, w, b)
    s = torch.zeros(8, 8).double()
    early, late = [], []
    for t in range(40):
        u = b[t] * (v[t] - s.T @ k[t])
        early.append(s.T @ q[t])
        s = w[t] * s + torch.outer(k[t], u)
        late.append(s.T @ q[t])
    assert rel(torch.stack(early), want) > 1e-2
    assert rel(torch.stack(late), want) > 1e-2
    _, half = plain.delta_scan(q[:20], k[:20], v[:20], w[:20], b[:20])
    parts = plain.delta_scan(q[20:], k[20:], v[20:], w[20:], b[20:], half)[0]
    assert rel(parts, want[20:]) < 1e-12
    lost = plain.delta_scan(q[20:], k[20:], v[20:], w[20:], b[20:])[0]
    assert rel(lost[:2], want[20:22]) > 1e-2
    taps = torch.randn(8, 3, generator=g).double()
    conv = plain.causal_conv(v, taps)
    assert rel(plain.causal_conv(v[20:], taps)[:2], conv[20:22]) > 1e-2
    assert torch.allclose(plain.causal_conv(v[18:], taps)[2:], conv[20:])
    assert torch.allclose(conv[0], taps[:, 2] * v[0])


def test_recurrence_sizes_are_checked():
    for args, what in (((32, 4, 3, 8, 8, 4, EPS), "groups"),
                       ((32, 4, 2, 8, 8, 9, EPS), "tokens"),
                       ((32, 4, 2, 300, 8, 4, EPS), "channels")):
        with pytest.raises(ValueError, match=what):
            GatedDelta(*args)
    with pytest.raises(ValueError, match="parts"):
        StateSpace(32, 2, 8, 8, 1, 4, 3, EPS)


@ALL
def test_both_mixers_side_by_side(device, dtype, tol):
    m, n, width = cases.parallel(), 70, 36
    st = random_state(cases.parallel_shapes(m, width), 3)
    h = inputs(n, width, 3)
    want = plain.parallel(h.double(), double(st), m, EPS)
    args, kw = attention_args(m["left"], width, EPS)
    r = m["right"]
    mod = ParallelMixer(
        width, GroupedAttention(*args, **kw), 0.5, StateSpace(
            width, r["heads"], r["vdim"], r["state"], r["groups"], r["conv"],
            r["norm_groups"], EPS), 0.5, norm_outputs=True)
    assert mod.shapes() == cases.parallel_shapes(m, width)
    mod.pack(st.__getitem__)

    def summed(mod, x, batch, cache):
        s = torch.zeros_like(x, dtype=torch.float32)
        lm.add_branches(s, None, mod.branches(x, batch, cache), mod.scale, [],
                        width, EPS, x.dtype)
        return s

    for portions in ([n], portions_of(n, [1]), portions_of(n, [33, 2])):
        assert rel(run_mixer(mod, h, portions, device, dtype,
                             forward=summed), want) < tol


# --------------------------------------------------------------------- #
# whole models through the engine
# --------------------------------------------------------------------- #
def setup(name, seed, dtype):
    """bf16 runs take weights that amplify rounding less"""
    cfg = cases.CONFIGS[name]()
    return cfg, cases.weights(cfg, seed, 2.5 if dtype == torch.float32
                              else 0.7)


@MODEL
@pytest.mark.parametrize("name", sorted(cases.CONFIGS))
def test_prompt_against_plain(device, dtype, tol, name, tmp_path):
    cfg, st = setup(name, 11, dtype)
    eng = engine(cfg, st, tmp_path, name_of(dtype), device)
    toks = tokens_for(cfg, 150, 1)
    want = plain.forward(cfg, st, toks)
    for portions in ([150], [1] * 150, portions_of(150, [2]),
                     portions_of(150, [64, 5, 1, 1, 33]),
                     portions_of(150, [9, 7])):
        got = feed_in_portions(eng, toks, portions)
        assert error(got, want) < tol, portions[:4]
    assert eng.allocator.available == 64 and eng.state_slots.available == 4


@MODEL
@pytest.mark.parametrize("name", ["mixed", "aligned"])
def test_stream_after_every_layer(device, dtype, tol, name, tmp_path):
    cfg, st = setup(name, 2, dtype)
    eng = engine(cfg, st, tmp_path, name_of(dtype), device)
    toks = tokens_for(cfg, 40, 3)
    want, got = [], []
    plain.forward(cfg, st, toks, collect=want)
    for lay in eng.model.layers:
        lay.register_forward_hook(
            lambda mod, args, out: got.append(args[0].clone()))
    feed_in_portions(eng, toks, [40])
    assert len(got) == len(want) == len(cfg["layers"])
    for g, w in zip(got, want):
        assert g.dtype == torch.float32
        assert rel(g[:, :cfg["width"]], w) < tol


def test_faults_between_layers_are_told_apart():
    cfg = cases.CONFIGS["mixed"]()
    st = cases.weights(cfg, 2)
    toks = tokens_for(cfg, 40, 3)
    want = plain.forward(cfg, st, toks)
    for k in ("l0.norm2", "l0.mix.left.out", "l3.mix.right.out",
              "l0.mix.left.sink", "l1.mix.dt_bias", "l3.mix.right.D",
              "l1.mix.norm", "l0.mlp.act", "l0.mix.right.conv.b"):
        assert error(plain.forward(cfg, dict(st, **{k: st[k] + 1.0}), toks),
                     want) > 0.003, k


@MODEL
@pytest.mark.parametrize("name", sorted(cases.CONFIGS))
def test_mixed_batches_and_reuse(device, dtype, tol, name, tmp_path):
    """Unequal requests come, pause, go; portions beside single tokens; the
    pool is small enough that pages and slots are used again. Every logit
    equals that of the request alone."""
    cfg, st = setup(name, 5, dtype)
    eng = engine(cfg, st, tmp_path, name_of(dtype), device, blocks=70)
    requests = []
    for i, n in enumerate([97, 3, 41, 66, 1, 58, 30, 2, 75]):
        toks = tokens_for(cfg, n, 100 + i)
        requests.append((toks, plain.forward(cfg, st, toks)))
    assert mixed_batches_error(eng, requests, seed=8) < 2 * tol
    assert eng.allocator.available == 70 and eng.state_slots.available == 4


@MODEL
def test_long_decoding(device, dtype, tol, tmp_path):
    cfg, st = setup("mixed", 6, dtype)
    eng = engine(cfg, st, tmp_path, name_of(dtype), device, blocks=130)
    toks = tokens_for(cfg, 400, 4)
    want = plain.forward(cfg, st, toks)
    got = feed_in_portions(eng, toks, [5] + [1] * 395)
    assert error(got, want) < tol


@pytest.mark.parametrize("device,dtype,tol", [CPU, GPU32])
@pytest.mark.parametrize("chunk,blocks", [(64, 120), (7, 120), (16, 20)],
                         ids=["whole", "portions", "preempted"])
def test_greedy_generation(device, dtype, tol, chunk, blocks, tmp_path):
    """the framework's own scheduler and sampling, also when prompts are cut
    and when sequences are preempted and start again"""
    cfg, st = setup("mixed", 7, dtype)
    eng = engine(cfg, st, tmp_path, name_of(dtype), device,
                 blocks=blocks, slots=3, prefill_chunk=chunk,
                 max_model_len=130)
    prompts = [tokens_for(cfg, n, 50 + n) for n in (31, 2, 17, 40, 9)]
    got = generate(eng, prompts, 15)
    for p, g in zip(prompts, got):
        want, lead = greedy(lambda t: plain.forward(cfg, st, t), p, 15)
        assert lead > 1e-4  # rounding cannot change a choice
        assert g == want
    if blocks == 20:
        assert eng.stats["preemptions"] > 0
    assert eng.allocator.available == blocks
    assert eng.state_slots.available == 3


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", ["bfloat16", "float32"])
@pytest.mark.parametrize("name", ["mixed", "aligned"])
def test_decode_graph_replays_equal_eager(dtype, name, tmp_path):
    """many replays, other work and other batch sizes between them"""
    cfg = cases.CONFIGS[name]()
    st = cases.weights(cfg, 9)
    runs = []
    for graphs in (True, False):
        eng = engine(cfg, st, tmp_path, dtype, "cuda:0",
                     decode_graphs=graphs)
        seqs = [open_sequence(eng) for _ in range(3)]
        toks = [tokens_for(cfg, 60, 20 + i) for i in range(3)]
        out = [eng.feed([(s, t[:9], [8]) for s, t in zip(seqs, toks)]).cpu()]
        for k in range(9, 60):
            use = [0, 1, 2] if k % 5 else [0]
            if k % 5 == 0:
                x = torch.randn(512, 512, device="cuda:0")
                (x @ x).sum().item()
            rows = eng.feed([(seqs[i], [toks[i][k]],
                              [0] if k % 3 else []) for i in use])
            out.append(rows.cpu().clone())
            if k % 5 == 0:
                out.append(eng.feed([(seqs[i], [toks[i][k]], [0])
                                     for i in (1, 2)]).cpu().clone())
        runs.append(torch.cat(out).float())
        assert (eng.stats["graph_replays"] > 40) == graphs
    assert torch.isfinite(runs[0]).all()
    assert (runs[0] - runs[1]).abs().max() <= 1e-5 * runs[1].abs().max()


@MODEL
def test_embeddings_leave_running_sequences_alone(device, dtype, tol,
                                                  tmp_path):
    cfg, st = setup("mixed", 10, dtype)
    eng = engine(cfg, st, tmp_path, name_of(dtype), device)
    toks = tokens_for(cfg, 50, 5)
    want = plain.forward(cfg, st, toks)
    s = open_sequence(eng)
    eng.feed([(s, toks[:30], [])])
    prompts = [tokens_for(cfg, n, n) for n in (12, 1, 20)]
    got = eng._embed_sync({"mode": "embed", "prompts": prompts,
                           "normalize": False})
    for p, g in zip(prompts, got):
        col = []
        plain.forward(cfg, st, p, collect=col)
        hid = (plain.over_rms(col[-1], cfg["norm"]["eps"])
               * st["final.norm"].double()).mean(0)
        assert rel(torch.tensor(g), hid) < tol
    got = eng.feed([(s, toks[30:], list(range(20)))])
    assert error(got, want[30:]) < tol


# --------------------------------------------------------------------- #
# configuration, loading, trace runner
# --------------------------------------------------------------------- #
def test_model_folder_selects_the_family(tmp_path):
    from clearml_serving_amd.engines.llm.engine import LlmEngineConfig
    from clearml_serving_amd.models import build_model, list_archs

    cfg = cases.CONFIGS["mixed"]()
    path = write_model(cfg, cases.weights(cfg), tmp_path / "m")
    ec = LlmEngineConfig.from_aux(path, {"max_num_seqs": 2})
    assert ec.arch == "nelovik" and ec.model_config == cfg
    assert "nelovik" in list_archs()
    model = build_model({"arch": "nelovik", "config": cfg,
                         "weights": ec.weights, "dtype": "float32"})
    assert model.cfg.vocab_size == cfg["vocab"]
    assert model.checkpoint_shapes() == cases.shapes(cfg)


def test_presets_build():
    from clearml_serving_amd.models import nelovik

    for raw in nelovik.PRESETS.values():
        nelovik.NelovikConfig(raw)
    model = nelovik.nelovik()
    model.init_random()
    model.finalize()


def test_bad_checkpoints_and_configs_are_refused(tmp_path):
    cfg = cases.CONFIGS["mixed"]()
    st = cases.weights(cfg)
    for change in (lambda s: s.pop("l1.mlp.act"),
                   lambda s: s.pop("l1.mix.dt_bias"),
                   lambda s: s.pop("l0.mix.left.q.b"),
                   lambda s: s.pop("l0.mix.right.out"),
                   lambda s: s.update(extra=s["embed"].clone()),
                   lambda s: s.update({"l0.norm1": s["embed"][0, :3]
                                       .clone()})):
        bad = dict(st)
        change(bad)
        with pytest.raises(ValueError, match="checkpoint"):
            engine(cfg, bad, tmp_path)
    # what belongs to a feed-forward that is not there does no harm
    engine(cfg, dict(st, **{"l2.norm2": st["l2.norm1"].clone()}), tmp_path)
    for change, what in (
            (lambda c: c["layers"][1]["mlp"].update(kind="other"), "mlp"),
            (lambda c: c["layers"][1].update(type="other"), "mixer"),
            (lambda c: c["layers"][1]["mixer"].update(kv_heads=3), "heads"),
            (lambda c: c["layers"][0]["mixer"]["left"]["rot"].update(dims=7),
             "rotated")):
        bad = json.loads(json.dumps(cfg))
        change(bad)
        with pytest.raises(ValueError, match=what):
            engine(bad, st, tmp_path)


@pytest.mark.parametrize("option", [
    {"quantization": "fp8"}, {"kv_dtype": "fp8"},
    {"enable_prefix_caching": True}, {"speculative": {"method": "ngram"}}])
def test_options_without_a_mechanism_are_refused(option, tmp_path):
    cfg = cases.CONFIGS["mixed"]()
    with pytest.raises(ValueError, match="does not support"):
        engine(cfg, cases.weights(cfg), tmp_path, **option)


@MODEL
def test_trace_runner_in_process(device, dtype, tol, tmp_path):
    from clearml_serving_amd.engines.llm import trace

    cfg, st = setup("mixed", 12, dtype)
    path = write_model(cfg, st, tmp_path / "m")
    out = str(tmp_path)
    a, b = tokens_for(cfg, 30, 1), tokens_for(cfg, 7, 2)
    eng = trace.make_engine(trace._parse([
        "--model", path, "--dtype", name_of(dtype), "--out", out,
        "--max-tokens", "128", "--device", device]))
    steps = []
    lines = io.StringIO("\n".join(json.dumps(x) for x in trace_lines(a, b)))
    trace.run(eng, lines, out, steps.append)
    assert steps == [0, 1, 2, 3]
    check_trace(out, cfg["vocab"],
                *(plain.forward(cfg, st, t) for t in (a, b)), tol)


def test_trace_runner_program(tmp_path):
    """bin/trace_run chooses the family by config.json"""
    cfg, st = setup("windows", 13, torch.float32)
    path = write_model(cfg, st, tmp_path / "m")
    a, b = tokens_for(cfg, 30, 1), tokens_for(cfg, 7, 2)
    lines = "".join(json.dumps(x) + "\n" for x in trace_lines(a, b))
    p = subprocess.run(
        [os.path.join(REPO, "bin", "trace_run"), "--model", path, "--dtype",
         "float32", "--out", str(tmp_path), "--max-tokens", "128",
         "--device", "cpu"], input=lines, capture_output=True, text=True,
        timeout=120)
    assert p.returncode == 0, p.stderr[-2000:]
    assert [x for x in p.stdout.splitlines() if x.startswith("done ")] == [
        "done {}".format(i) for i in range(4)]
    check_trace(str(tmp_path), cfg["vocab"],
                *(plain.forward(cfg, st, t) for t in (a, b)), 2e-5)


@pytest.mark.gpu
def test_bf16_generation_is_the_same_alone_and_together(tmp_path):
    """greedy, through the scheduler, in bf16: graphs, buckets and prompt
    portions change nothing where the choice is clear"""
    cfg, st = setup("aligned", 14, torch.bfloat16)
    st["embed"] = st["embed"] * 6
    st["head"] = st["embed"].roll(-1, 0)  # the next token is clear
    prompts = [tokens_for(cfg, n, 60 + n) for n in (33, 1, 12)]
    eng = engine(cfg, st, tmp_path, "bfloat16", "cuda:0", slots=3,
                 prefill_chunk=10, max_model_len=128)
    together = generate(eng, prompts, 12)
    clear = 0
    for p, g in zip(prompts, together):
        eng = engine(cfg, st, tmp_path, "bfloat16", "cuda:0", slots=3,
                     max_model_len=128)
        want, lead = greedy(lambda t: plain.forward(cfg, st, t), p, 12)
        if lead > 0.5:
            clear += 1
            assert generate(eng, [p], 12) == [g]
            assert g == want
    assert clear
