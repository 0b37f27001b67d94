"""Engines, sequences and comparisons that the tests of all token-batch
families share."""

import asyncio
import json
import os
import random

import torch
from safetensors.torch import save_file


def name_of(dtype):
    return {torch.float32: "float32", torch.bfloat16: "bfloat16"}[dtype]


def padded(x, n):
    out = torch.zeros(*x.shape[:-1], n, dtype=x.dtype)
    out[..., :x.shape[-1]] = x
    return out


def rel(got, want):
    d = (got.double().cpu() - want.double()).abs().max()
    return (d / want.abs().max().clamp(min=1e-6)).item()


def error(got, want):
    """per row: rms difference over the rms of all wanted logits"""
    d = got.double().cpu() - want
    d = d - d.mean(-1, keepdim=True)
    return (d.pow(2).mean(-1).sqrt() / want.pow(2).mean().sqrt()).max().item()


def portions_of(n, sizes):
    """cut n into the given sizes, cycled"""
    out, i = [], 0
    while n:
        k = min(sizes[i % len(sizes)], n)
        out.append(k)
        n -= k
        i += 1
    return out


def tokens_for(cfg, n, seed):
    r = random.Random(seed)
    return [r.randrange(cfg["vocab"]) for _ in range(n)]


def engine(cfg, state, tmp_path, dtype="float32", device="cpu", blocks=64,
           block_size=4, slots=4, **kw):
    from clearml_serving_amd.engines.llm.engine import (LlmEngine,
                                                        LlmEngineConfig)

    path = os.path.join(str(tmp_path), "model.safetensors")
    save_file({k: v.contiguous() for k, v in state.items()}, path)
    kw.setdefault("max_model_len", blocks * block_size)
    e = LlmEngine(LlmEngineConfig(
        arch=cfg["architecture"].lower(), model_config=cfg, weights=path,
        dtype=dtype, device=device, num_kv_blocks=blocks,
        block_size=block_size, max_num_seqs=slots, **kw))
    e.start()
    return e


def write_model(cfg, st, folder):
    os.makedirs(folder, exist_ok=True)
    with open(os.path.join(folder, "config.json"), "w") as f:
        json.dump(cfg, f)
    save_file({k: v.contiguous() for k, v in st.items()},
              os.path.join(folder, "model.safetensors"))
    return str(folder)


def open_sequence(eng, name="s"):
    from clearml_serving_amd.engines.llm.engine import (SamplingParams,
                                                        Sequence)

    s = Sequence(name, [], SamplingParams())
    eng.open_sequence(s)
    return s


def feed_in_portions(eng, tokens, portions):
    """one sequence, cut as given -> logits of every token (CPU, float64)"""
    s = open_sequence(eng)
    out, at = [], 0
    for n in portions:
        part = tokens[at:at + n]
        out.append(eng.feed([(s, part, list(range(len(part))))])
                   .double().cpu())
        at += n
    assert at == len(tokens)
    eng.close_sequence(s)
    return torch.cat(out)


def mixed_batches_error(eng, requests, seed):
    """requests: (tokens, wanted logits). They come, pause and go, portions
    beside single tokens, at most four at a time -> worst row error"""
    r = random.Random(seed)
    left, live, worst = list(requests), [], 0.0
    while left or live:
        while left and len(live) < 4:
            toks, want = left.pop(0)
            live.append([open_sequence(eng), toks, want, 0])
        todo = [x for x in live if r.random() < 0.8] or live[:1]
        r.shuffle(todo)
        entries, spans = [], []
        for x in todo:
            n = min(r.choice([1, 1, 1, 2, 3, 13, 40]), len(x[1]) - x[3])
            want = sorted(r.sample(range(n), r.randint(0, n)))
            entries.append((x[0], x[1][x[3]:x[3] + n], want))
            spans.append((x, [x[3] + w for w in want]))
            x[3] += n
        logits = eng.feed(entries).cpu()
        at = 0
        for x, places in spans:
            if places and x[2][places].abs().max() > 0:
                worst = max(worst, error(logits[at:at + len(places)],
                                         x[2][places]))
            at += len(places)
        assert at == len(logits)
        for x in [x for x in live if x[3] == len(x[1])]:
            eng.close_sequence(x[0])
            live.remove(x)
    return worst


def greedy(forward, prompt, n):
    """forward(tokens) -> logits of every token. -> greedy tokens, smallest
    lead of a chosen logit over the runner-up"""
    ids, lead = list(prompt), float("inf")
    for _ in range(n):
        top = forward(ids)[-1].topk(2)
        lead = min(lead, (top.values[0] - top.values[1]).item())
        ids.append(int(top.indices[0]))
    return ids[len(prompt):], lead


def generate(eng, prompts, n):
    from clearml_serving_amd.engines.llm.engine import SamplingParams

    async def one(ids):
        seq = await eng.add_request(ids, SamplingParams(
            temperature=0.0, max_tokens=n, ignore_eos=True))
        out = []
        while True:
            item = await seq.stream.get()
            assert not item.get("error"), item
            out.extend(item["token_ids"])
            if item["finished"]:
                return out

    async def main():
        out = await asyncio.gather(*[one(p) for p in prompts])
        # the step that finished the last request also gives back its pages
        await asyncio.sleep(0.05)
        return out

    return asyncio.new_event_loop().run_until_complete(main())


def trace_lines(toks_a, toks_b):
    """20 or more tokens and 7 tokens as steps of a trace"""
    yield {"step": 0, "entries": [
        {"id": "a", "tokens": toks_a[:20], "want": [0, 19]},
        {"id": "b", "tokens": toks_b[:2], "want": []}], "end": []}
    yield {"step": 1, "entries": [
        {"id": "b", "tokens": toks_b[2:], "want": [0, 4]},
        {"id": "a", "tokens": toks_a[20:21], "want": [0]}], "end": ["b"]}
    yield {"step": 2, "entries": [
        {"id": "a", "tokens": toks_a[21:], "want": []}], "end": ["a"]}
    yield {"step": 3, "entries": [
        {"id": "c", "tokens": toks_b[:1], "want": [0]}], "end": ["c"]}


def check_trace(out, vocab, wa, wb, tol):
    """wa, wb: wanted logits of both requests of trace_lines"""
    import numpy as np

    for step, want in ((0, wa[[0, 19]]),
                       (1, torch.stack([wb[2], wb[6], wa[20]])),
                       (3, wb[:1])):
        got = np.fromfile(os.path.join(out, "{}.f32".format(step)),
                          dtype="<f4").reshape(-1, vocab)
        assert error(torch.from_numpy(got), want) < tol
    assert not os.path.exists(os.path.join(out, "2.f32"))
