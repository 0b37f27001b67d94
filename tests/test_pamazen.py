"""Pamazen against a plain implementation of its equations
(tests/helpers/pamazen_plain.py): each mechanism alone, then whole models
through the engine -- prompts cut in every way, mixed batches, reused pages
and slots, greedy generation. Each case runs on the CPU reference operations
and, marked gpu, on the kernels in 32-bit and bf16."""

import io
import json
import math
import os
import subprocess
import sys

import pytest
import torch

sys.path.insert(0, os.path.join(os.path.dirname(__file__), "helpers"))

import pamazen_cases as cases  # noqa: E402
import pamazen_plain as plain  # noqa: E402
from lm_cases import (check_trace, engine, error,  # noqa: E402
                      feed_in_portions, generate, greedy,
                      mixed_batches_error, name_of, open_sequence, padded,
                      portions_of, rel, tokens_for, trace_lines, write_model)

from clearml_serving_amd.engines.llm.token_batch import TokenBatch  # noqa: E402
from clearml_serving_amd.models.mixers import (DeltaRule,  # noqa: E402
                                               ExpertMlp, GroupedAttention,
                                               GroupedAttentionMixer,
                                               ParallelMixer)
from clearml_serving_amd.ops import delta, hyper, lm  # noqa: E402

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


# --------------------------------------------------------------------- #
# streams
# --------------------------------------------------------------------- #
@ALL
@pytest.mark.parametrize("streams", [1, 2, 3, 4, 5, 6, 7, 8])
@pytest.mark.parametrize("width", [44, 300, 2080])
def test_streams_around_a_sublayer(device, dtype, tol, width, streams):
    """one step: the output goes to all streams, the next sublayer's norm"""
    n, eps, m, wp = 4, 1e-2, 0.7, lm.pad32(width)
    g = torch.Generator().manual_seed(streams)
    x = torch.randn(n, streams, width, generator=g)
    o = torch.randn(n, width, generator=g).to(dtype)
    x[2] *= 1e-2  # eps matters here
    o[2] *= 1e-2
    w = {k: torch.randn(s, generator=g).to(torch.bfloat16) for k, s in (
        ("in", (streams,)), ("out", (streams,)), ("mix", (streams,) * 2))}
    nxt, gain = (torch.randn(s, generator=g).to(torch.bfloat16)
                 for s in ((streams,), ()))
    want = torch.stack(plain.out_of(list(x.double().unbind(1)), o.double(),
                                    double(w), m), 1)
    after = gain.double() * plain.over_rms(plain.into(
        list(want.unbind(1)), {"in": nxt.double()}), eps)
    coef = hyper.step_coef(w["mix"], w["out"], m, nxt, gain).to(device)
    for last in (False, True):
        xs = padded(x, wp).to(device)
        h = hyper.step(padded(o, wp).to(device), xs, coef, width, eps, last)
        assert h.dtype == dtype and rel(h[:, :width], after) < max(tol, 1e-5)
        # the streams are 32-bit whatever the product type is
        if not last:
            assert xs.dtype == torch.float32
            assert rel(xs[..., :width], want) < 1e-5
        if wp > width:
            assert h[:, width:].abs().max() == 0
            assert xs[..., width:].abs().max() == 0
    if streams > 1:  # [from, to], not the other way round
        turned = dict(double(w), mix=w["mix"].double().T)
        assert rel(torch.stack(plain.out_of(
            list(x.double().unbind(1)), o.double(), turned, m), 1),
            want) > 0.05


@ALL
def test_rows_and_identities_into_the_streams(device, dtype, tol):
    """what a mixture leaves: rows anywhere, a weight each, and slots that
    stand for the sublayer's input"""
    n, slots, width, s = 6, 3, 40, 2
    g = torch.Generator().manual_seed(2)
    rows = padded(torch.randn(n * slots, width, generator=g), 64).to(dtype)
    pos = torch.randperm(n * slots, generator=g).view(n, slots).int()
    pos[0, 1] = pos[3, 0] = pos[3, 2] = pos[5] = -1
    share = torch.rand(n, slots, generator=g)
    skip = padded(torch.randn(n, width, generator=g), 64).to(dtype)
    x = padded(torch.randn(n, s, width, generator=g), 64)
    picked = torch.where((pos < 0)[..., None], skip.double()[:, None],
                         rows.double()[pos.long().clamp(min=0)])
    y = (picked * share.double()[..., None]).sum(1)
    w = {"mix": torch.eye(s), "out": torch.tensor([1.0, -2.0])}
    want = torch.stack(plain.out_of(list(x.double().unbind(1)), y,
                                    double(w), 1.0), 1)
    xs = x.to(device)
    coef = hyper.step_coef(w["mix"], w["out"], 1.0, torch.ones(s),
                           torch.tensor(1.0)).to(device)
    hyper.step(rows.to(device), xs, coef, width, 1e-5, False,
               (pos.to(device), share.to(device)), skip.to(device))
    assert rel(xs, want) < 1e-5


@ALL
def test_embedding_and_output_cap(device, dtype, tol):
    vocab, width, wp, eps, s = 9, 40, 64, 1e-3, 3
    g = torch.Generator().manual_seed(3)
    table = torch.randn(vocab, width, generator=g).to(dtype)
    w_in, gain = torch.randn(s, generator=g), torch.tensor(-1.5)
    toks = torch.tensor([3, 0, 8, 3])
    x, h = hyper.embed(toks.to(device), padded(table, wp).to(device),
                       hyper.entry_coef(w_in, gain).to(device), s, width, eps)
    x0 = table.double()[toks]
    assert x.dtype == torch.float32
    assert rel(x[..., :width], x0[:, None].expand(-1, s, -1)) == 0
    assert rel(h[:, :width], -1.5 * plain.over_rms(
        w_in.double().sum() * x0, eps)) < max(tol, 1e-5)
    z = (30 * torch.randn(5, 64, generator=g)).to(dtype)
    z[0, 0] = 1e-3
    got = hyper.soft_cap(z.to(device), 37, 7.5)
    assert got.dtype == torch.float32 and got.shape == (5, 37)
    assert rel(got, plain.soft_cap(z.double()[:, :37], 7.5)) < 1e-5


# --------------------------------------------------------------------- #
# running one mixer on a sequence
# --------------------------------------------------------------------- #
def random_state(shapes, seed, sharp=2.5):
    g = torch.Generator().manual_seed(seed)
    return {k: cases.random_tensor(k, s, g, sharp).to(torch.bfloat16)
            for k, s in shapes.items()}


def caches_for(mod, n_pages, block_size, slots, device, dtype):
    """filled with what earlier owners may have left"""
    def make(kind, *dims):
        if kind == "both":
            return tuple(make(*d) for d in dims)
        if kind == "paged":
            return torch.full((n_pages, block_size, dims[0]), 3.0,
                              dtype=dtype, device=device)
        return (torch.full((slots, *dims[0]), 2.0, device=device),)
    return make(*mod.cache_layout())


def run_mixer(mod, h, portions, device, dtype, block_size=4, absorb_max=None,
              pages=None, carry=None):
    """one sequence through a mixer in portions -> [n, width] float64.
    ``carry``: per token, the first mixing layer's values"""
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
        c = {} if carry is None else {
            "values": carry[at:at + k].to(dtype).to(device)}
        out.append(mod(x, batch, cache, c).double().cpu())
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
# attention over everything
# --------------------------------------------------------------------- #
def attention_of(m, width):
    r = m["rot"]
    return GroupedAttentionMixer(
        width, m["heads"], m["kv_heads"], m["dim"], m["vdim"], m["scale"],
        rot=(r["base"], r["dims"], r["scaling"]["factor"]), sink="one",
        v_mix=m["v_mix"])


ATTN_SIZES = [
    dict(), dict(heads=20, kv=1, dim=40, rot=34, vdim=70),
    dict(heads=1, kv=1, dim=2, rot=2, vdim=1, factor=1.0),
    dict(heads=6, kv=3, dim=96, rot=96, vdim=130, base=1e6),
    dict(heads=4, kv=4, dim=200, rot=64, vdim=64, v_mix=False),
    dict(heads=4, kv=2, dim=64, rot=32, vdim=200),
]


@ALL
@FORMS
@pytest.mark.parametrize("size", range(len(ATTN_SIZES)))
def test_attention_sizes(device, dtype, tol, absorb_max, size):
    skip_expanded_in_32_bit(absorb_max, device, dtype)
    m = cases.attn(**ATTN_SIZES[size])
    m["scale"] = m["dim"] ** -0.5
    n, width = 200, 36
    st = random_state(cases.attention_shapes(m, width), size)
    g = torch.Generator().manual_seed(size)
    h = torch.randn(n, width, generator=g).to(torch.bfloat16)
    first = None
    if m["v_mix"]:
        first = torch.randn(n, m["kv_heads"], m["vdim"], generator=g) \
            .to(torch.bfloat16)
    want, own = plain.attention(
        h.double(), double(st), m, None if first is None else first.double())
    mod = attention_of(m, width)
    mod.pack(st.__getitem__)
    carry = None if first is None else padded(
        first, lm.pad32(m["vdim"])).reshape(n, -1)
    pages = [3 * (i % 5) + i // 5 for i in range(15)]  # in no order
    for portions in ([n], portions_of(n, [131, 2, 1, 40])):
        got = run_mixer(mod, h, portions, device, dtype, 16, absorb_max,
                        pages, carry)
        assert rel(got, want) < tol
    if first is not None:  # the first such layer's own values are unmixed
        assert rel(run_mixer(mod, h, [n], device, dtype, 16, absorb_max,
                             pages), plain.attention(
            h.double(), double(st), m, None)[0]) < tol


def needle(st, h, m, key, query, strong=9.0):
    """the query at `query` scores the key at `key` far above all others, by
    the first dimension that is not rotated; values tell the keys apart"""
    d = m["rot"]["dims"] if "rot" in m else 0
    h[:, :2] = 0
    h[key, 0] = h[query, 1] = 12.0
    for k in ("q", "k"):
        st[k] *= 0.05
        st[k][:, :2] = 0
    if "v" in st:
        st["v"][:, :2] = 0
    for a in range(m["heads"]):
        st["q"][a * m["dim"] + d] = 0
        st["q"][a * m["dim"] + d, 1] = strong
    for a in range(m["kv_heads"]):
        st["k"][a * m["dim"] + d] = 0
        st["k"][a * m["dim"] + d, 0] = strong


@ALL
@FORMS
@pytest.mark.parametrize("key,query", [(0, 299), (3, 299), (4, 298),
                                       (64, 130), (127, 129), (298, 299),
                                       (299, 299)])
def test_one_key_stands_out(device, dtype, tol, absorb_max, key, query):
    """far away, at page and tile borders, the query itself"""
    skip_expanded_in_32_bit(absorb_max, device, dtype)
    m, n, width = cases.attn(v_mix=False), 300, 36
    st = random_state(cases.attention_shapes(m, width), 5)
    h = torch.randn(n, width, generator=torch.Generator().manual_seed(1)) \
        .to(torch.bfloat16)
    needle(st, h, m, key, query, 1.0)
    want, _ = plain.attention(h.double(), double(st), m, None)
    mod = attention_of(m, width)
    mod.pack(st.__getitem__)
    for portions in ([n], [query] + [1] * (n - query) if query else [n],
                     portions_of(n, [67, 2])):
        got = run_mixer(mod, h, portions, device, dtype,
                        absorb_max=absorb_max)
        assert rel(got, want) < tol
    # the oracle without that key is told apart
    h2 = h.clone()
    h2[key, 0] = 0
    without, _ = plain.attention(h2.double(), double(st), m, None)
    assert rel(without[query], want[query]) > 5 * tol


def test_frequencies_and_sinks():
    m = cases.attn(base=500.0, rot=6, factor=3.0)
    mod = attention_of(m, 36)
    mod.finalize()
    assert torch.allclose(mod.attn.rot.inv_freq.double(),
                          plain.frequencies(m["rot"]), rtol=1e-6)
    # with one key: e^s / (1 + e^s)
    w = plain.weigh(torch.tensor([[0.0]]), torch.tensor([[True]]),
                    torch.tensor(0.0))
    assert math.isclose(w.item(), 0.5)


# --------------------------------------------------------------------- #
# windows with kept first tokens, capped scores, learned sinks
# --------------------------------------------------------------------- #
class WindowOnly(ParallelMixer):
    """the left side alone"""

    def __init__(self, width, m, eps):
        super().__init__(width, window_of(m, width, eps), 1.0,
                         DeltaRule(width, 1, 1, eps, 1), 0.0)


def window_of(m, width, eps):
    return GroupedAttention(
        width, m["heads"], m["kv_heads"], m["dim"], m["vdim"], m["scale"],
        eps, window=m["mask"]["size"], keep=m["mask"]["keep_first"],
        cap=m["softcap"], qk_norm=True, values_are_keys=True, sink="learned")


def window_state(m, width, seed):
    st = random_state(cases.attention_shapes(m, width, True), seed)
    both = {"left." + k: v for k, v in st.items()}
    both.update({"right." + k: v for k, v in random_state(
        cases.delta_shapes({"heads": 1, "dim": 1}, width, 1), 0).items()})
    return st, both


WINDOWS = [
    dict(), dict(heads=1, kv=1, dim=1, size=1, keep=0),
    dict(heads=20, kv=1, dim=33, size=64, keep=1),
    dict(heads=4, kv=4, dim=128, size=65, keep=70, cap=25.0),
    dict(heads=6, kv=3, dim=64, size=100, keep=17, cap=2.0),
    dict(heads=2, kv=2, dim=200, size=33, keep=32),
]


@ALL
@FORMS
@pytest.mark.parametrize("size", range(len(WINDOWS)))
def test_window_attention(device, dtype, tol, absorb_max, size):
    skip_expanded_in_32_bit(absorb_max, device, dtype)
    m = cases.left(**WINDOWS[size])
    n, width = 230, 36
    st, both = window_state(m, width, size)
    h = torch.randn(n, width, generator=torch.Generator()
                    .manual_seed(size)).to(torch.bfloat16)
    h[1] *= 1e-2  # eps of the head norms matters here
    want = plain.window_attention(h.double(), double(st), m, EPS)
    mod = WindowOnly(width, m, EPS)
    mod.pack(both.__getitem__)
    pages = [3 * (i % 5) + i // 5 for i in range(15)]
    for portions in ([n], portions_of(n, [131, 2, 1, 40])):
        got = run_mixer(mod, h, portions, device, dtype, 16, absorb_max,
                        pages)
        assert rel(got, want) < tol
    # the oracle with one thing wrong is told apart
    wrong = dict(double(st), sink=st["sink"].double() - 3.0)
    assert rel(plain.window_attention(h.double(), wrong, m, EPS),
               want) > 1e-2


@ALL
@FORMS
@pytest.mark.parametrize("size,keep", [(11, 3), (64, 5), (70, 0)])
def test_window_edges(device, dtype, tol, absorb_max, size, keep):
    """a key that stands out, just inside and just outside of the window and
    of the kept tokens, in prompts and decoding"""
    skip_expanded_in_32_bit(absorb_max, device, dtype)
    m = cases.left(heads=4, kv=2, dim=20, size=size, keep=keep, cap=30.0,
                   scale=0.8)
    n, width = 160, 36
    for query in (n - 1, n - 30):
        for key, seen in ((query - size + 1, True), (query - size, False),
                          (keep - 1, True), (keep, False)):
            if key < 0:
                continue
            st, both = window_state(m, width, 4)
            h = torch.randn(n, width, generator=torch.Generator()
                            .manual_seed(key)).to(torch.bfloat16)
            w = {k: both["left." + k] for k in st}
            needle(w, h, m, key, query, 4.0)
            for k in ("q.norm", "k.norm", "sink"):
                w[k].abs_()
            both.update({"left." + k: v for k, v in w.items()})
            want = plain.window_attention(h.double(), double(w), m, EPS)
            mod = WindowOnly(width, m, EPS)
            mod.pack(both.__getitem__)
            for portions in ([n], [query - 3] + [1] * (n - query + 3),
                             portions_of(n, [67, 2])):
                got = run_mixer(mod, h, portions, device, dtype,
                                absorb_max=absorb_max)
                assert rel(got, want) < tol
            other = dict(m, mask={"size": size + (1 if not seen and
                                                  key != keep else 0),
                                  "keep_first": keep + (key == keep)})
            if key == keep - 1:
                other["mask"]["keep_first"] = keep - 1
            elif seen:
                other["mask"]["size"] = size - 1
            off = plain.window_attention(h.double(), double(w), other, EPS)
            assert rel(off[query], want[query]) > 3 * tol


# --------------------------------------------------------------------- #
# delta rule
# --------------------------------------------------------------------- #
class DeltaOnly(DeltaRule):
    """as a mixer of its own"""

    def finalize(self):
        super().finalize()
        self.inp = self.inp.to(self.w2)
        self.o = self.o.to(self.w2)

    def pack(self, get):
        w = lm.pad32(self.width)
        self.inp = torch.zeros(self.cols, w)
        self.o = torch.zeros(w, self.out_cols)
        self.pack_in(self.inp, get)
        self.pack_out(self.o, get)
        self.pack_own(get)

    def cache_layout(self):
        return self.state_layout()

    def forward(self, h, batch, cache, carry):
        z = h @ self.inp.T
        out = h.new_empty(h.shape[0], self.out_cols)
        self.scan(z, batch, cache[0], out)
        return out @ self.o.T


@ALL
@pytest.mark.parametrize("heads,dim,rank", [
    (2, 24, 5), (1, 1, 1), (3, 64, 32), (1, 33, 70), (2, 96, 64),
    (1, 128, 40), (1, 150, 3), (1, 256, 32)])
def test_delta_rule(device, dtype, tol, heads, dim, rank):
    m, n, width = {"heads": heads, "dim": dim}, 90, 36
    st = random_state(cases.delta_shapes(m, width, rank), dim)
    h = torch.randn(n, width, generator=torch.Generator().manual_seed(dim)) \
        .to(torch.bfloat16)
    want = plain.delta_rule(h.double(), double(st), m, EPS)
    mod = DeltaOnly(width, heads, dim, EPS, rank)
    mod.pack(st.__getitem__)
    for portions in ([n], portions_of(n, [1]),
                     portions_of(n, [17, 2, 1, 16, 3])):
        assert rel(run_mixer(mod, h, portions, device, dtype), want) < tol


@ALL
@pytest.mark.parametrize("heads,dim,chunk", [
    (2, 24, 1), (1, 64, 2), (2, 96, 1), (1, 128, 3), (1, 150, 1),
    (1, 256, 2)])
def test_delta_rule_in_chunks(device, dtype, tol, heads, dim, chunk,
                              monkeypatch):
    """long portions are cut, and walked from the states in front of the
    chunks; portions end inside, at and right behind a chunk's end"""
    monkeypatch.setattr(delta, "chunk_tiles", lambda *a: chunk)
    m, n, width = {"heads": heads, "dim": dim}, 600, 36
    st = random_state(cases.delta_shapes(m, width, 8), dim)
    h = torch.randn(n, width, generator=torch.Generator().manual_seed(dim)) \
        .to(torch.bfloat16)
    want = plain.delta_rule(h.double(), double(st), m, EPS)
    mod = DeltaOnly(width, heads, dim, EPS, 8)
    mod.pack(st.__getitem__)
    for portions in ([n], [128, 2, 192, 65, 1, 212], [5, 64, 531]):
        assert rel(run_mixer(mod, h, portions, device, dtype), want) < tol


def test_which_portions_are_cut():
    assert delta.chunk_tiles(0, 0, 4) == 0  # none
    assert delta.chunk_tiles(4, 1, 4) == 0  # short
    assert delta.chunk_tiles(4000, 64, 16) == 0  # enough of them
    for tiles, seqs, heads in ((128, 1, 16), (128, 4, 16), (2000, 1, 1)):
        assert 3 <= delta.chunk_tiles(tiles, seqs, heads) < tiles / seqs


def test_delta_oracle_tells_faults_apart():
    """both terms read the old state; a lost state, a wrong key shows"""
    g = torch.Generator().manual_seed(0)
    r, k, v = (torch.randn(40, 8, generator=g).double() for _ in range(3))
    w, a = (torch.rand(40, 8, generator=g).double() for _ in range(2))
    want, _ = plain.delta_scan(r, k, v, w, a)
    s = torch.zeros(8, 8).double()
    late = []
    for t in range(40):
        s = w[t][:, None] * s
        u = k[t] / torch.sqrt(k[t] @ k[t] + 1e-6)
        s = s - torch.outer(a[t] * u, u @ s) + torch.outer(k[t], v[t])
        late.append(s.T @ r[t])
    assert rel(torch.stack(late), want) > 1e-2
    _, half = plain.delta_scan(r[:20], k[:20], v[:20], w[:20], a[:20])
    parts = plain.delta_scan(r[20:], k[20:], v[20:], w[20:], a[20:], half)[0]
    assert rel(parts, want[20:]) < 1e-12
    lost = plain.delta_scan(r[20:], k[20:], v[20:], w[20:], a[20:])[0]
    assert rel(lost[:2], want[20:22]) > 1e-2


@ALL
def test_both_mixers_side_by_side(device, dtype, tol):
    m, n, width = cases.parallel(), 70, 36
    shapes = {"left." + k: s for k, s in cases.attention_shapes(
        m["left"], width, True).items()}
    shapes.update({"right." + k: s for k, s in cases.delta_shapes(
        m["right"], width, 5).items()})
    st = random_state(shapes, 3)
    h = torch.randn(n, width, generator=torch.Generator().manual_seed(3)) \
        .to(torch.bfloat16)
    want = plain.parallel(h.double(), double(st), m, EPS)
    mod = ParallelMixer(width, window_of(m["left"], width, EPS), 0.8,
                        DeltaRule(width, 2, 24, EPS), 1.3)
    mod.fit(st.__getitem__)  # the rank is the checkpoint's
    mod.pack(st.__getitem__)
    for portions in ([n], portions_of(n, [1]), portions_of(n, [33, 2])):
        assert rel(run_mixer(mod, h, portions, device, dtype), want) < tol


# --------------------------------------------------------------------- #
# experts
# --------------------------------------------------------------------- #
def routed(p, top, real):
    """ids per slot from an ExpertPlan's tile list (GPU) or rows (CPU)"""
    plan = p.plan.cpu().tolist()
    expert_of = {}
    if p.share.is_cuda:
        for k in range(plan[0]):
            e, first, count = plan[1 + 3 * k:4 + 3 * k]
            assert 1 <= count <= p.rows
            for r in range(first, first + count):
                assert r not in expert_of
                expert_of[r] = e
    else:
        expert_of = dict(enumerate(plan))
    return [[expert_of[r] if r >= 0 else -1 for r in row]
            for row in p.pos.cpu().tolist()]


@ALL
@pytest.mark.parametrize("experts,identity,top,groups,shared", [
    (6, 2, 2, (4, 3), 1), (5, 1, 3, (2, 1), 2), (1, 0, 1, (1, 1), 0),
    (3, 3, 2, (6, 2), 1), (62, 2, 8, (8, 4), 1), (90, 6, 16, (4, 1), 3),
    (128, 0, 4, (16, 16), 1)])
@pytest.mark.parametrize("n", [1, 37])
def test_routing(device, dtype, tol, experts, identity, top, groups, shared,
                 n):
    g = torch.Generator().manual_seed(experts)
    width, out = 64, experts + identity
    h = torch.randn(n, width, generator=g).to(dtype)
    w = (torch.randn(out + (shared > 0), width, generator=g) * 0.2).to(dtype)
    # steps that no score can bridge, most of them negative
    c = 1.5 * torch.randint(-3, 1, (out,), generator=g).float()
    r = {"experts": experts, "identity": identity, "top": top,
         "groups": {"count": groups[0], "keep": groups[1]}}
    ids, share = plain.route(h.double(), w[:out].double(), c.double(), r)
    how = lm.Routing(top, True, groups[0], groups[1], identity, shared)
    p = lm.moe_route(h.to(device), w.to(device), how, 16, c.to(device))
    if shared:
        gate = plain.sigmoid(h.double() @ w[out].double())[:, None]
        share = torch.cat([share, gate.expand(-1, shared)], 1)
    want = [[e if e < experts else -1 for e in row]
            + list(range(experts, experts + shared)) for row in ids.tolist()]
    got = routed(p, top, experts)
    # experts may come in any order
    for t in range(n):
        key = sorted(range(top + shared), key=lambda k: (got[t][k],
                                                         p.share[t, k].item()))
        ref = sorted(range(top + shared), key=lambda k: (want[t][k],
                                                         share[t, k].item()))
        assert [got[t][k] for k in key] == [want[t][k] for k in ref]
        assert rel(p.share[t].cpu()[key], share[t][ref]) < 1e-4


def test_left_out_groups_count_as_minus_infinity():
    """all choice scores negative: a group left out must not win with 0"""
    r = {"experts": 4, "identity": 0, "top": 2,
         "groups": {"count": 2, "keep": 1}}
    c = torch.tensor([-5.0, -6.0, -2.0, -9.0])
    h, w = torch.ones(1, 32), torch.zeros(4, 32)
    ids, share = plain.route(h.double(), w.double(), c.double(), r)
    assert ids.tolist() == [[2, 3]] and share.tolist() == [[0.25, 0.25]]
    p = lm.moe_route(h, w, lm.Routing(2, True, 2, 1), 16, c)
    assert routed(p, 2, 4) == [[2, 3]]


@ALL
@pytest.mark.parametrize("width,kw", [
    (44, {}), (40, dict(experts=5, top=3, ff=24, identity=1, groups=(2, 1),
                        shared=60)),
    (33, dict(experts=3, top=3, ff=1, identity=0, groups=(1, 1), shared=1)),
    (128, dict(experts=8, top=4, ff=64, identity=4, groups=(4, 2),
               shared=192)),
    (64, dict(experts=6, top=2, ff=192, identity=6, groups=(2, 2),
              shared=64))])
def test_mixture(device, dtype, tol, width, kw):
    """token counts that make tiles of several sizes"""
    mlp = cases.moe(**kw)
    r = mlp["router"]
    st = random_state(cases.moe_shapes(mlp, width), width)
    st["correction"] = 1.5 * torch.randint(
        -1, 2, st["correction"].shape,
        generator=torch.Generator().manual_seed(1)).to(torch.bfloat16)
    mod = ExpertMlp(width, mlp["expert"]["ff"], r["experts"], r["top"],
                    act="silu", gated=True, correction=True,
                    groups=(r["groups"]["count"], r["groups"]["keep"]),
                    identity=r["identity"], shared_ff=mlp["shared"]["ff"])
    assert mod.shapes() == cases.moe_shapes(mlp, width)
    mod.pack(st.__getitem__)
    mod = mod.to(device).to(dtype)
    mod.finalize()
    big = torch.randn(400, width, generator=torch.Generator()
                      .manual_seed(7)).to(torch.bfloat16)
    want = plain.mixture(big.double(), double(st), mlp)
    for n in (1, 2, 10, 40, 130, 400):
        x = padded(big[:n], lm.pad32(width)).to(dtype).to(device)
        out, (pos, share) = mod(x)
        got = torch.where((pos < 0)[..., None], x.float()[:, None],
                          out.float()[pos.long().clamp(min=0)])
        got = (got * share[..., None]).sum(1).cpu()
        assert rel(got[:, :width], want[:n]) < tol
    # the oracle with one thing wrong is told apart
    for change in (lambda s: s.update({"shared.sg": 0 * s["shared.sg"]}),
                   lambda s: s.update({k: s[k.replace("gate", "up")]
                                       for k in s if k[0] == "e"
                                       and k.endswith("gate")})):
        wrong = dict(double(st))
        change(wrong)
        assert rel(plain.mixture(big.double(), wrong, mlp), want) > 1e-3


# --------------------------------------------------------------------- #
# whole models through the engine
# --------------------------------------------------------------------- #
def setup(name, seed, dtype):
    """bf16 runs take weights that amplify rounding less, and whose routing
    does not hang on it"""
    c = cases.CONFIGS[name]()
    if dtype == torch.float32:
        return cases.public(c), cases.weights(c, seed)
    return cases.public(c), cases.weights(c, seed, 0.7, decided=True)


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
def test_streams_after_every_layer(device, dtype, tol, name, tmp_path):
    cfg, st = setup(name, 2, dtype)
    eng = engine(cfg, st, tmp_path, name_of(dtype), device)
    toks = tokens_for(cfg, 40, 3)
    want, got = [], []
    plain.forward(cfg, st, toks, collect=want)
    for lay in eng.model.layers:
        lay.last = False  # write the streams of the last layer too
        lay.register_forward_hook(
            lambda mod, args, out: got.append(args[0].clone()))
    feed_in_portions(eng, toks, [40])
    assert len(got) == len(want) == len(cfg["layers"])
    for g, w in zip(got, want):
        assert g.dtype == torch.float32
        assert rel(g.sum(1)[:, :cfg["width"]], w) < tol


def test_faults_between_layers_are_told_apart():
    c = cases.CONFIGS["mixed"]()
    cfg, st = cases.public(c), cases.weights(c, 2)
    toks = tokens_for(cfg, 40, 3)
    want = plain.forward(cfg, st, toks)
    changes = {"residual_mult": 1.0, "logit_softcap": 20.0}
    for k, v in changes.items():
        assert error(plain.forward(dict(cfg, **{k: v}), st, toks),
                     want) > 0.01
    turned = dict(st, **{"l1.mlp.correction":
                         st["l1.mlp.correction"].flip(0)})
    assert error(plain.forward(cfg, turned, toks), want) > 0.003
    for k in ("l3.mix.vmix", "l1.mix.left.sink", "l1.mix.right.w0",
              "l0.norm2"):
        assert error(plain.forward(cfg, dict(st, **{k: st[k] + 1.0}), toks),
                     want) > 0.003, k
    # the first mixing layer's own factor is unused
    assert torch.equal(plain.forward(
        cfg, dict(st, **{"l2.mix.vmix": st["l2.mix.vmix"] + 1}), toks), want)


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
    c = cases.CONFIGS[name]()
    cfg, st = cases.public(c), cases.weights(c, 9, decided=True)
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

    c = cases.CONFIGS["mixed"]()
    cfg = cases.public(c)
    path = write_model(cfg, cases.weights(c), tmp_path / "m")
    ec = LlmEngineConfig.from_aux(path, {"max_num_seqs": 2})
    assert ec.arch == "pamazen" and ec.model_config == cfg
    assert "pamazen" in list_archs()
    model = build_model({"arch": "pamazen", "config": cfg,
                         "weights": ec.weights, "dtype": "float32"})
    assert model.cfg.vocab_size == cfg["vocab"]
    assert model.checkpoint_shapes() == cases.shapes(c)


def test_presets_build():
    from clearml_serving_amd.models import pamazen

    for raw in pamazen.PRESETS.values():
        pamazen.PamazenConfig(raw)
    model = pamazen.pamazen()
    model.init_random()
    model.finalize()


def test_bad_checkpoints_and_configs_are_refused(tmp_path):
    c = cases.CONFIGS["mixed"]()
    cfg, st = cases.public(c), cases.weights(c)
    for change in (lambda s: s.pop("l1.mlp.e4.down"),
                   lambda s: s.pop("l1.mix.right.w1"),
                   lambda s: s.pop("l0.hc2.mix"),
                   lambda s: s.update(extra=s["embed"].clone()),
                   lambda s: s.update({"l0.norm1": s["embed"][0, :3]
                                       .clone()})):
        bad = dict(st)
        change(bad)
        with pytest.raises(ValueError, match="checkpoint"):
            engine(cfg, bad, tmp_path)
    # what belongs to a feed-forward that is not there does no harm, nor does
    # a factor of values that are not mixed
    engine(cfg, dict(st, **{"l2.norm2": st["l2.norm1"].clone(),
                            "l2.hc2.in": st["l2.hc1.in"].clone(),
                            "l0.mix.vmix": st["l0.norm1"].clone()}), tmp_path)
    for change, what in (
            (lambda c: c["layers"][1]["mlp"].update(kind="other"), "mlp"),
            (lambda c: c["layers"][1].update(type="other"), "mixer"),
            (lambda c: c.update(streams=9), "streams"),
            (lambda c: c["layers"][3]["mixer"].update(vdim=11), "values"),
            (lambda c: c["layers"][1]["mlp"]["router"].update(top=7),
             "experts")):
        bad = json.loads(json.dumps(cfg))
        change(bad)
        with pytest.raises(ValueError, match=what):
            engine(bad, st, tmp_path)


@pytest.mark.parametrize("option", [
    {"quantization": "fp8"}, {"kv_dtype": "fp8"},
    {"enable_prefix_caching": True}, {"speculative": {"method": "ngram"}}])
def test_options_without_a_mechanism_are_refused(option, tmp_path):
    c = cases.CONFIGS["mixed"]()
    with pytest.raises(ValueError, match="does not support"):
        engine(cases.public(c), cases.weights(c), tmp_path, **option)


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
    st["head"] = st["embed"].roll(-1, 0)  # the next token is clear
    prompts = [tokens_for(cfg, n, 60 + n) for n in (33, 1, 12)]
    eng = engine(cfg, st, tmp_path, "bfloat16", "cuda:0", slots=3,
                 prefill_chunk=10, max_model_len=128)
    together = generate(eng, prompts, 12)
    for p, g in zip(prompts, together):
        eng = engine(cfg, st, tmp_path, "bfloat16", "cuda:0", slots=3,
                     max_model_len=128)
        want, lead = greedy(lambda t: plain.forward(cfg, st, t), p, 12)
        assert lead < 0.5 or generate(eng, [p], 12) == [g]
        assert lead < 0.5 or g == want
