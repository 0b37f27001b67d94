"""Prefill and decode throughput of the token-batch families (Nelovik, Pamazen,
Kakipel, Bimipel) beside llama at equal size, random weights, through the LLM
engine's own forwards.

    python bench.py --workload lm [--lm-size 300m,1b,4k] [--lm-model ...]

One JSON line per model, size and phase. Prefill: prompts of --lm-prompt
tokens, one forward of up to 8192 tokens. Decode: --lm-batch sequences behind
prompts of that length, hipGraph-replayed steps.
"""

import gc
import json
import time

import torch

SIZES = {
    # size -> model -> (preset, overrides)
    "300m": {"nelovik": ("nelovik-300m", {}),
             "pamazen": ("pamazen-300m", {}),
             "kakipel": ("kakipel-300m", {}), "bimipel": ("bimipel-300m", {}),
             "llama": ("llama-3-8b", dict(
                 vocab_size=32000, hidden=1024, layers=12, heads=16,
                 kv_heads=4, intermediate=3584))},
    "1b": {"nelovik": ("nelovik-1b", {}),
           "pamazen": ("pamazen-1b", {}),
           "kakipel": ("kakipel-1b", {}), "bimipel": ("bimipel-1b", {}),
           "llama": ("llama-3-1b", {})},
    # few layers, as wide as an 8B model's
    "4k": {"nelovik": ("nelovik-4k", {}),
           "pamazen": ("pamazen-4k", {}),
           "kakipel": ("kakipel-4k", {}), "bimipel": ("bimipel-4k", {}),
           "llama": ("llama-3-8b", dict(vocab_size=32000, layers=6,
                                        intermediate=12288))},
}


def _params(model):
    seen = {}
    for p in model.parameters():
        seen[p.data_ptr()] = p.numel()
    return sum(seen.values())


def _engine(kind, size, batch, max_len):
    from clearml_serving_amd.engines.llm.engine import (LlmEngine,
                                                        LlmEngineConfig)

    preset, over = SIZES[size][kind]
    blocks = max(batch, 1) * (-(-max_len // 16) + 1)
    cfg = LlmEngineConfig(
        arch=kind, preset=preset, overrides=dict(over),
        max_num_seqs=batch, max_model_len=max_len, num_kv_blocks=blocks,
        device="cuda:0" if torch.cuda.is_available() else "cpu")
    eng = LlmEngine(cfg)
    eng.start()
    return eng


def _timed(fn, iters, warmup=3):
    for _ in range(warmup):
        fn()
    torch.cuda.synchronize()
    t0 = time.perf_counter()
    for _ in range(iters):
        fn()
    torch.cuda.synchronize()
    return (time.perf_counter() - t0) / iters


def _plans(eng, prompts, prompt_len):
    """prompts at block ranges of their own -> (prefill fn, decode fn)"""
    bs = eng.cfg.block_size
    per = -(-(prompt_len + 2) // bs)
    n = len(prompts)
    blocks = [list(range(i * per, (i + 1) * per)) for i in range(n)]
    nxt = [p[0] for p in prompts]
    if eng.token_batch:
        def plan(idx, tokens, start):
            return {"tokens": tokens, "starts": [start] * len(idx),
                    "blocks": [blocks[i] for i in idx],
                    "state_slots": list(idx),
                    "want": [[len(t) - 1] for t in tokens]}

        def prefill(idx):
            return eng._exec_batch(plan(idx, [prompts[i] for i in idx], 0))

        def decode():
            return eng._exec_batch(plan(range(n), [[t] for t in nxt],
                                        prompt_len))
    else:
        def slot(i, p):
            return blocks[i][p // bs] * bs + p % bs

        slots = [[slot(i, p) for p in range(prompt_len)] for i in range(n)]

        def prefill(idx):
            return eng._exec_prefill({
                "prompts": [prompts[i] for i in idx],
                "slots": [slots[i] for i in idx]})

        def decode():
            return eng._exec_decode({
                "tokens": nxt, "positions": [prompt_len] * n,
                "slots": [slot(i, prompt_len) for i in range(n)],
                "seq_lens": [prompt_len + 1] * n, "blocks": blocks})
    return prefill, decode


def run(sizes, models, prompt_len=2048, batches=(1, 16, 64), iters=20,
        phases=("prefill", "decode")):
    for size in sizes:
        for kind in models:
            top = max(batches) if "decode" in phases else 4
            eng = _engine(kind, size, max(top, 4), prompt_len + 64)
            vocab = eng.model_config.vocab_size
            gen = torch.Generator().manual_seed(7)
            prompts = [torch.randint(1, vocab, (prompt_len,), generator=gen)
                       .tolist() for _ in range(max(top, 4))]
            base = {"model": kind, "size": size, "dtype": "bf16",
                    "params_m": round(_params(eng.model) / 1e6),
                    "data": "synthetic", "prompt": prompt_len}
            group = max(1, 8192 // prompt_len)
            if "prefill" in phases:
                prefill, _ = _plans(eng, prompts, prompt_len)
                idx = list(range(min(group, len(prompts))))
                dt = _timed(lambda: prefill(idx), iters)
                print(json.dumps({
                    **base, "phase": "prefill", "batch": len(idx),
                    "ms": round(dt * 1e3, 3),
                    "tok_s": round(len(idx) * prompt_len / dt)}), flush=True)
            if "decode" in phases:
                for b in batches:
                    prefill, decode = _plans(eng, prompts[:b], prompt_len)
                    for i in range(0, b, group):
                        prefill(list(range(i, min(i + group, b))))
                    dt = _timed(decode, iters * 3)
                    print(json.dumps({
                        **base, "phase": "decode", "batch": b,
                        "ms": round(dt * 1e3, 3),
                        "tok_s": round(b / dt)}), flush=True)
            eng.stop()
            del eng
            gc.collect()
            torch.cuda.empty_cache()
