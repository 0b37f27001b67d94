"""Bimipel against a plain implementation of its equations
(tests/helpers/bimipel_plain.py): each mechanism alone, then whole models
through the engine -- prompts cut in every way, mixed batches, reused pages
and slots, greedy generation. Each case runs on the CPU reference operations
and, marked gpu, on the kernels in 32-bit and bf16."""

import asyncio
import io
import json
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

sys.path.insert(0, os.path.join(os.path.dirname(__file__), "helpers"))

import bimipel_cases as cases  # noqa: E402
import bimipel_plain as plain  # noqa: E402
from lm_cases import (check_trace, engine, error,  # noqa: E402
                      feed_in_portions, generate, greedy,
                      mixed_batches_error, name_of, open_sequence, padded,
                      portions_of, rel, tokens_for, trace_lines, write_model)

from clearml_serving_amd.engines.llm.token_batch import TokenBatch  # noqa: E402
from clearml_serving_amd.models.mixers import (GatedMlp,  # noqa: E402
                                               LatentAttention, RgLru)
from clearml_serving_amd.ops import lm  # noqa: E402

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


# --------------------------------------------------------------------- #
# mechanisms alone
# --------------------------------------------------------------------- #
@ALL
def test_norm_on_output_and_residual(device, dtype, tol):
    n, width, eps = 5, 44, 1e-2
    g = torch.Generator().manual_seed(1)
    o = torch.randn(n, width, generator=g).to(dtype)
    b, w = (torch.randn(width, generator=g).to(dtype) for _ in range(2))
    x = torch.randn(n, width, generator=g)
    o[2] *= 1e-2  # eps matters here
    b0 = torch.zeros_like(b)
    for bias, used in ((b, b), (None, b0)):
        want = x.double() + plain.norm_zero_centred(
            o.double() + used.double(), w.double(), eps)
        xs = padded(x, 64).to(device)
        h = lm.post_norm_add(
            padded(o, 64).to(device),
            None if bias is None else padded(bias, 64).to(device),
            padded(w, 64).to(device), xs, width, eps)
        # the stream is 32-bit whatever the product type is
        assert rel(xs[:, :width], want) < 1e-5
        assert h.dtype == dtype and rel(h[:, :width], want) < max(tol, 1e-5)
        assert xs[:, width:].abs().max() == 0
    rows = torch.tensor([3, 0], dtype=torch.int32)
    got = lm.output_norm(padded(x, 64).to(device), rows.to(device),
                         padded(w, 64).to(device), width, eps, 0.3)
    want = 0.3 * plain.norm_zero_centred(x.double()[[3, 0]], w.double(), eps)
    assert rel(got[:, :width], want) < max(tol, 1e-5)


@ALL
@pytest.mark.parametrize("width", [2080, 4224, 8224])
def test_norm_wide_rows(device, dtype, tol, width):
    g = torch.Generator().manual_seed(2)
    o = torch.randn(3, width, generator=g).to(dtype)
    w = torch.randn(width, generator=g).to(dtype)
    x = torch.randn(3, width, generator=g)
    want = x.double() + plain.norm_zero_centred(o.double(), w.double(), 1e-5)
    xs = x.clone().to(device)
    lm.post_norm_add(o.to(device), None, w.to(device), xs, width, 1e-5)
    assert rel(xs, want) < 1e-5


@ALL
def test_feed_forward(device, dtype, tol):
    width, ff, n = 44, 20, 37
    g = torch.Generator().manual_seed(3)
    mod = GatedMlp(width, ff)
    st = {k: torch.randn(s, generator=g).to(torch.bfloat16)
          for k, s in mod.shapes().items()}
    mod.pack(st.__getitem__)
    mod = mod.to(device).to(dtype)
    h = torch.randn(n, width, generator=g).to(torch.bfloat16)
    got = mod(padded(h, 64).to(dtype).to(device)).float().cpu() \
        + mod.down_b.float().cpu()
    want = plain.feed_forward(h.double(),
                              {k: v.double() for k, v in st.items()})
    assert rel(got[:, :width], want) < tol
    assert got[:, width:].abs().max() == 0


def attention_setup(m, width, n, seed, eps=1e-5, strong=2.5):
    g = torch.Generator().manual_seed(seed)
    mod = LatentAttention(width, m["heads"], m["dim"], m["rot_dim"],
                          m["vdim"], m["kv_rank"], m["scale"],
                          m["mask"]["size"], m["rot"]["base"],
                          m["rot"]["dims"], eps)
    st = {}
    for k, s in mod.shapes().items():
        t = torch.randn(s, generator=g)
        if k == "q":
            t = strong * t
        if len(s) == 2:
            t = t * s[-1] ** -0.5
        elif k == "dkv.norm":
            t = 1 + 0.2 * t
        st[k] = t.to(torch.bfloat16)
    h = torch.randn(n, width, generator=g).to(torch.bfloat16)
    return mod, st, h


def run_attention(mod, st, h, portions, device, dtype, block_size=4,
                  absorb_max=None, pages=None):
    """one sequence through the layer in portions -> [n, width] float64"""
    mod.pack(st.__getitem__)
    mod = mod.to(device).to(dtype)
    mod.finalize()
    n = h.shape[0]
    need = -(-n // block_size)
    pages = pages or list(range(need))
    cache = torch.full((max(pages) + 1, block_size, mod.row), 3.0,
                       dtype=dtype, device=device)
    out, at = [], 0
    for k in portions:
        _, batch, _ = TokenBatch.build(
            {"tokens": [[0] * k], "starts": [at], "blocks": [pages],
             "state_slots": [0], "want": [[]]}, block_size, device,
            tile=64, absorb_max=absorb_max, windows=[mod.window])
        x = padded(h[at:at + k], lm.pad32(mod.width)).to(dtype).to(device)
        out.append(mod(x, batch, cache).double().cpu())
        at += k
    return torch.cat(out)[:, :mod.width]


def want_attention(st, h, m, eps=1e-5):
    w = {k: v.double() for k, v in st.items()}
    x = h.double()
    c, kr = plain.latent_and_rotated_key(x, w, m, eps)
    return plain.latent_attention(x, w, m, c, kr)


# absorbed: every token scores the cache rows; expanded: prompts rebuild keys
FORMS = pytest.mark.parametrize("absorb_max", [None, 1],
                                ids=["absorbed", "expanded"])
ATTN_SIZES = [
    dict(heads=3, dim=12, rot=6, vdim=10, rank=20, window=7),
    dict(heads=17, dim=40, rot=34, vdim=70, rank=100, window=70),
    dict(heads=1, dim=1, rot=2, vdim=1, rank=1, window=1),
    dict(heads=2, dim=96, rot=32, vdim=130, rank=200, window=150),
    dict(heads=2, dim=150, rot=64, vdim=200, rank=300, window=40),
    dict(heads=4, dim=64, rot=32, vdim=64, rank=520, window=500),
]


@ALL
@FORMS
@pytest.mark.parametrize("size", range(len(ATTN_SIZES)))
def test_attention_sizes(device, dtype, tol, absorb_max, size):
    if absorb_max is not None and device != "cpu" \
            and dtype == torch.float32:
        pytest.skip("prompts take the absorbed form in 32-bit")
    m = cases.attn(**ATTN_SIZES[size])
    m["scale"] = (m["dim"] + m["rot_dim"]) ** -0.5
    n = 200
    mod, st, h = attention_setup(m, 36, n, seed=size)
    want = want_attention(st, h, m)
    for portions in ([n], portions_of(n, [131, 2, 1, 40])):
        got = run_attention(mod, st, h, portions, device, dtype,
                            block_size=16, absorb_max=absorb_max)
        assert rel(got, want) < tol


def needle_setup(m, width, n, key, query, seed=5):
    """the query at `query` scores the key at `key` far above all others"""
    mod, st, h = attention_setup(m, width, n, seed, strong=0.05)
    # input coordinate 0 is set at the key only and drives latent dimension
    # 0; coordinate 1 is set at the query only; dimension 0 of every head's
    # unrotated query and key carries them
    h[:, :2] = 0
    h[key, 0] = 12.0
    h[query, 1] = 12.0
    for k in ("dkv", "q"):
        st[k][:, :2] = 0
    st["dkv"][0] = 0
    st["dkv"][0, 0] = 4.0
    st["uv"][:, 0] *= 6
    d = m["dim"] + m["rot_dim"]
    for a in range(m["heads"]):
        st["uk"][a * m["dim"]] = 0
        st["uk"][a * m["dim"], 0] = 3.0
        st["q"][a * d, 1] = 3.0
    return mod, st, h


@ALL
@FORMS
@pytest.mark.parametrize("window", [1, 5, 16, 17, 64, 130])
def test_window_edges(device, dtype, tol, absorb_max, window):
    """A key at the last visible distance and one step beyond, at several
    places relative to pages and tiles, in prompts and decoded alone. The
    plain form with a window off by one must be told apart."""
    if absorb_max is not None and device != "cpu" \
            and dtype == torch.float32:
        pytest.skip("prompts take the absorbed form in 32-bit")
    m = cases.attn(heads=2, dim=16, rot=8, vdim=12, rank=24, window=window,
                   scale=0.5)
    for query in (window + 31, window + 64, window + 3):
        for dist in (window - 1, window):
            key = query - dist
            n = query + 1
            mod, st, h = needle_setup(m, 36, n, key, query)
            want = want_attention(st, h, m)
            got = run_attention(mod, st, h, [n], device, dtype,
                                absorb_max=absorb_max)
            assert rel(got[query], want[query]) < tol
            got = run_attention(mod, st, h, [n - 1, 1], device, dtype,
                                absorb_max=absorb_max)
            assert rel(got[query], want[query]) < tol
            if window > 1:
                for wrong in (window - 1, window + 1):
                    if (dist < wrong) == (dist < window):
                        continue
                    off = want_attention(st, h,
                                         {**m, "mask": {"size": wrong}})
                    assert rel(off[query], want[query]) > 3 * tol


@ALL
@FORMS
def test_sink_counts_once_unscaled(device, dtype, tol, absorb_max):
    if absorb_max is not None and device != "cpu" \
            and dtype == torch.float32:
        pytest.skip("prompts take the absorbed form in 32-bit")
    m = cases.attn(heads=3, dim=16, rot=8, vdim=12, rank=24, window=9,
                   scale=0.2)
    for sinks in ([2.2] * 3, [4.0, -30.0, 60.0]):
        mod, st, h = attention_setup(m, 36, 70, seed=9, strong=1.0)
        st["sink"] = torch.tensor(sinks, dtype=torch.bfloat16)
        want = want_attention(st, h, m)
        got = run_attention(mod, st, h, [33, 5, 1, 31], device, dtype,
                            absorb_max=absorb_max)
        assert rel(got, want) < tol
        if sinks[0] == 2.2:  # scaled, counted twice, left out
            for wrong in (m["scale"] * 2.2, 2.2 + np.log(2.0), -60.0):
                bad = dict(st, sink=torch.full((3,), wrong))
                assert rel(want_attention(bad, h, m), want) > 3 * tol


@ALL
def test_rotation_far_positions(device, dtype, tol):
    """positions in the tens of thousands keep their 32-bit angles"""
    g = torch.Generator().manual_seed(4)
    heads, dp, rp, cp, rot = 2, 32, 32, 32, 10
    pos = torch.tensor([0, 1, 999, 40000], dtype=torch.int32)
    qkv = torch.randn(4, heads * (dp + rp) + cp + rp, generator=g).to(dtype)
    ref = qkv.double()
    inv = (1000.0 ** (-2.0 * torch.arange(rot // 2).double() / rot)).float()
    cache = torch.zeros(3, 4, cp + rp, dtype=dtype).to(device)
    slots = torch.tensor([0, 5, 7, -1], dtype=torch.int32)
    q_abs = torch.zeros(2, heads, cp + rp, dtype=dtype).to(device)
    dev = qkv.clone().to(device)
    lm.latent_prep(dev, pos.to(device), slots.to(device),
                   lm.Rotary(inv.to(device)), heads, dp, rp, cp, 20, 1e-5,
                   torch.ones(cp, dtype=dtype).to(device), cache, q_abs)
    t = 1e-3 if dtype == torch.float32 else 2e-2
    q = ref[:, :heads * (dp + rp)].view(4, heads, dp + rp)
    want = torch.cat([plain.rotate_pairs(q[..., dp:dp + rot], pos, 1000.0),
                      q[..., dp + rot:]], -1)
    assert rel(q_abs[..., cp:], want[:2]) < t
    got = dev[:, :heads * (dp + rp)].view(4, heads, -1)[2:, :, dp:]
    assert rel(got, want[2:]) < t
    kr = ref[:, heads * (dp + rp) + cp:]
    want = torch.cat([plain.rotate_pairs(kr[:, :rot], pos, 1000.0),
                      kr[:, rot:]], -1)
    flat = cache.view(12, -1).double().cpu()
    assert rel(flat[[0, 5, 7], cp:], want[:3]) < t
    assert flat[[1, 2, 3, 4, 6, 8, 9, 10, 11]].abs().max() == 0


REC_SIZES = [(24, 3, 4), (20, 1, 1), (66, 2, 2), (7, 7, 3), (384, 2, 7),
             (320, 1, 4)]


def rec_setup(width, m, n, seed):
    g = torch.Generator().manual_seed(seed)
    mod = RgLru(width, m["width"], m["blocks"], m["conv"])
    st = {}
    for k, s in mod.shapes().items():
        t = torch.randn(s, generator=g)
        if k == "lam":
            t = -3 + 3 * t  # from nearly no memory to nearly no decay
        elif k != "conv" and len(s) > 1 and not k.endswith(".b"):
            t = t * s[-1] ** -0.5
        st[k] = t.to(torch.bfloat16)
    h = torch.randn(n, width, generator=g).to(torch.bfloat16)
    return mod, st, h


def run_rec(mod, st, h, portions, device, dtype, tile=64, slot=1):
    mod.pack(st.__getitem__)
    mod = mod.to(device).to(dtype)
    mod.finalize()
    # state left by somebody else: position 0 must not see it
    cache = (torch.full((3, mod.wp), 9.0).to(device),
             torch.full((3, mod.taps, mod.wp), 9.0, dtype=dtype).to(device))
    out, at = [], 0
    for k in portions:
        _, batch, _ = TokenBatch.build(
            {"tokens": [[0] * k], "starts": [at],
             "blocks": [list(range(-(-h.shape[0] // 4)))],
             "state_slots": [slot], "want": [[]]}, 4, device, tile=tile,
            absorb_max=None, windows=[])
        x = padded(h[at:at + k], lm.pad32(mod.width)).to(dtype).to(device)
        out.append(mod(x, batch, cache).double().cpu())
        at += k
    for c in cache:  # other slots are untouched
        assert (c[[0, 2]] == 9.0).all()
    return torch.cat(out)[:, :mod.width]


@ALL
@pytest.mark.parametrize("tile", [64, 16])
@pytest.mark.parametrize("size", REC_SIZES)
def test_recurrence(device, dtype, tol, size, tile):
    m = cases.rec(*size)
    n = 150
    mod, st, h = rec_setup(40, m, n, seed=sum(size))
    w = {k: v.double() for k, v in st.items()}
    want = plain.rglru(h.double(), w)
    if 128 * (lm.pad32(mod.bw) + 8) * dtype.itemsize > 160 * 1024:
        tile = 16
    for portions in ([n], [1] * n, portions_of(n, [2, 3, 1]),
                     portions_of(n, [65, 1, 17])):
        got = run_rec(mod, st, h, portions, device, dtype, tile=tile)
        assert rel(got, want) < tol
    # the oracle with one thing wrong is told apart
    wrong = dict(w, lam=w["lam"] + 0.7)
    assert rel(plain.rglru(h.double(), wrong), want) > tol


@ALL
def test_recurrence_long_memory(device, dtype, tol):
    """almost no decay: 1 - a^2 must not cancel, early tokens still count"""
    m = cases.rec(32, 1, 2)
    mod, st, h = rec_setup(32, m, 600, seed=3)
    st["lam"] = torch.full_like(st["lam"], -9.0)
    want = plain.rglru(h.double(), {k: v.double() for k, v in st.items()})
    for portions in ([600], portions_of(600, [100, 1])):
        assert rel(run_rec(mod, st, h, portions, device, dtype), want) < tol


# --------------------------------------------------------------------- #
# whole models through the engine
# --------------------------------------------------------------------- #
def model_weights(cfg, seed, dtype):
    """bf16 runs take weights that amplify rounding less"""
    return cases.weights(cfg, seed, 2.5 if dtype == torch.float32 else 0.7)


@MODEL
@pytest.mark.parametrize("name", sorted(cases.CONFIGS))
def test_prompt_against_plain(device, dtype, tol, name, tmp_path):
    cfg = cases.CONFIGS[name]()
    st = model_weights(cfg, 11, dtype)
    eng = engine(cfg, st, tmp_path, name_of(dtype), device)
    toks = tokens_for(cfg, 190, 1)
    want = plain.forward(cfg, st, toks)
    for portions in ([190], [1] * 190, portions_of(190, [2]),
                     portions_of(190, [64, 5, 1, 1, 33]),
                     portions_of(190, [9, 7])):
        got = feed_in_portions(eng, toks, portions)
        assert error(got, want) < tol, portions[:4]
    assert eng.allocator.available == 64 and eng.state_slots.available == 4


@MODEL
def test_residual_after_every_layer(device, dtype, tol, tmp_path):
    cfg = cases.CONFIGS["mixed"]()
    st = model_weights(cfg, 2, dtype)
    eng = engine(cfg, st, tmp_path, name_of(dtype), device)
    toks = tokens_for(cfg, 40, 3)
    want, got = [], []
    plain.forward(cfg, st, toks, collect=want)
    for lay in eng.model.layers:
        lay.register_forward_hook(
            lambda mod, args, out: got.append(args[0].clone()))
    feed_in_portions(eng, toks, [40])
    for g, w in zip(got, want):
        assert g.dtype == torch.float32
        assert rel(g[:, :cfg["width"]], w) < tol


@MODEL
@pytest.mark.parametrize("name", ["mixed", "recurrent_first"])
def test_mixed_batches_and_reuse(device, dtype, tol, name, tmp_path):
    """Unequal requests come, pause, go; portions beside single tokens; the
    pool is small enough that pages and slots are used again. Every logit
    equals that of the request alone."""
    cfg = cases.CONFIGS[name]()
    st = model_weights(cfg, 5, dtype)
    eng = engine(cfg, st, tmp_path, name_of(dtype), device, blocks=70)
    requests = []
    for i, n in enumerate([97, 3, 41, 66, 1, 58, 30, 2, 75]):
        toks = tokens_for(cfg, n, 100 + i)
        requests.append((toks, plain.forward(cfg, st, toks)))
    worst = mixed_batches_error(eng, requests, seed=8)
    assert worst < 2 * tol
    assert eng.allocator.available == 70 and eng.state_slots.available == 4


@MODEL
def test_long_decoding(device, dtype, tol, tmp_path):
    cfg = cases.CONFIGS["mixed"]()
    st = model_weights(cfg, 6, dtype)
    eng = engine(cfg, st, tmp_path, name_of(dtype), device, blocks=160)
    toks = tokens_for(cfg, 600, 4)
    want = plain.forward(cfg, st, toks)
    got = feed_in_portions(eng, toks, [5] + [1] * 595)
    assert error(got, want) < tol


@pytest.mark.parametrize("device,dtype,tol", [CPU, GPU32])
@pytest.mark.parametrize("chunk,blocks", [(64, 120), (7, 120), (16, 20)],
                         ids=["whole", "portions", "preempted"])
def test_greedy_generation(device, dtype, tol, chunk, blocks, tmp_path):
    """the framework's own scheduler and sampling, also when prompts are cut
    and when sequences are preempted and start again"""
    cfg = cases.CONFIGS["mixed"]()
    st = model_weights(cfg, 7, dtype)
    eng = engine(cfg, st, tmp_path, name_of(dtype), device,
                       blocks=blocks, slots=3, prefill_chunk=chunk,
                       max_model_len=130)
    prompts = [tokens_for(cfg, n, 50 + n) for n in (31, 2, 17, 40, 9)]
    got = generate(eng, prompts, 24)
    for p, g in zip(prompts, got):
        want, lead = greedy(lambda t: plain.forward(cfg, st, t), p, 24)
        assert lead > 1e-4  # rounding cannot change a choice
        assert g == want
    if blocks == 20:
        assert eng.stats["preemptions"] > 0
    assert eng.allocator.available == blocks
    assert eng.state_slots.available == 3


@pytest.mark.gpu
@pytest.mark.parametrize("dtype", ["bfloat16", "float32"])
def test_decode_graph_replays_equal_eager(dtype, tmp_path):
    """many replays, other work and other batch sizes between them"""
    cfg = cases.CONFIGS["mixed"]()
    st = cases.weights(cfg, seed=9)
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
    cfg = cases.CONFIGS["mixed"]()
    st = model_weights(cfg, 10, dtype)
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
        hid = plain.norm_zero_centred(col[-1], st["final.norm"].double(),
                                      cfg["norm"]["eps"]).mean(0)
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
    assert ec.arch == "bimipel" and ec.model_config == cfg
    assert ec.weights.endswith("model.safetensors")
    assert "bimipel" in list_archs()
    model = build_model({"arch": "bimipel", "config": cfg,
                         "weights": ec.weights, "dtype": "float32"})
    assert model.cfg.vocab_size == cfg["vocab"]
    # a config.json of another library's model is left alone
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump({"architectures": ["LlamaForCausalLM"]}, f)
    assert LlmEngineConfig.from_aux(path, {}).arch == "llama"


def test_bad_checkpoints_and_configs_are_refused(tmp_path):
    cfg = cases.CONFIGS["mixed"]()
    st = cases.weights(cfg)
    for change in (lambda s: s.pop("l0.mix.sink"),
                   lambda s: s.update(extra=s["embed"].clone()),
                   lambda s: s.update({"l0.norm1": s["embed"][0, :3].clone()})):
        bad = dict(st)
        change(bad)
        with pytest.raises(ValueError, match="checkpoint"):
            engine(cfg, bad, tmp_path)
    for src in (1, 2, 5):
        bad = cases.CONFIGS["mixed"]()
        bad["layers"][2]["mixer"]["kv_from"] = src
        with pytest.raises(ValueError, match="kv_from"):
            engine(bad, st, tmp_path)
    bad = cases.CONFIGS["mixed"]()
    bad["layers"][2]["mixer"]["rot"]["base"] = 9.0
    with pytest.raises(ValueError, match="rot"):
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

    cfg = cases.CONFIGS["mixed"]()
    st = cases.weights(cfg, seed=12)
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
    check_trace(out, cfg["vocab"], *(plain.forward(cfg, st, t)
                                      for t in (a, b)), tol)


def test_trace_runner_program(tmp_path):
    """bin/trace_run answers step by step on its pipe"""
    cfg = cases.CONFIGS["mixed"]()
    st = cases.weights(cfg, seed=13)
    path = write_model(cfg, st, tmp_path / "m")
    a, b = tokens_for(cfg, 30, 1), tokens_for(cfg, 7, 2)
    p = subprocess.Popen(
        [os.path.join(REPO, "bin", "trace_run"), "--model", path, "--dtype",
         "float32", "--out", str(tmp_path), "--max-tokens", "128",
         "--device", "cpu"], stdin=subprocess.PIPE, stdout=subprocess.PIPE,
        text=True)
    try:
        for step in trace_lines(a, b):
            p.stdin.write(json.dumps(step) + "\n")
            p.stdin.flush()
            while True:
                line = p.stdout.readline()
                assert line, "ended early"
                if line.strip() == "done {}".format(step["step"]):
                    break
        p.stdin.close()
        assert p.wait(timeout=60) == 0
    finally:
        p.kill()
    check_trace(str(tmp_path), cfg["vocab"],
                *(plain.forward(cfg, st, t) for t in (a, b)), 2e-5)


@pytest.mark.gpu
def test_bf16_generation_through_the_serving_adapter(tmp_path):
    """model folder -> registered endpoint -> completion"""
    from clearml_serving_amd.engines.llm.adapter import LlmPreprocessRequest
    from clearml_serving_amd.schemas import ModelEndpoint

    cfg = cases.config([cases.layer(cases.attn(), ff=36),
                        cases.layer(cases.rec())], vocab=300)
    path = write_model(cfg, cases.weights(cfg, seed=14), tmp_path / "m")

    class Request(LlmPreprocessRequest):
        def _get_local_model_file(self):
            return path

    req = Request(ModelEndpoint(
        engine_type="llm", serving_url="bim", model_id="bim-test",
        auxiliary_cfg={"max_num_seqs": 4, "max_model_len": 256}))

    async def main():
        body = {"prompt": "hello", "max_tokens": 6, "temperature": 0,
                "ignore_eos": True}
        return await asyncio.gather(*[req.process(dict(body), {})
                                      for _ in range(3)])

    outs = asyncio.new_event_loop().run_until_complete(main())
    assert all(o["tokens"] == 6 for o in outs)
    assert len({o["text"] for o in outs}) == 1
    req.shutdown()
