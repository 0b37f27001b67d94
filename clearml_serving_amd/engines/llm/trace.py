"""Replay a trace: feed given token ids to the LLM engine step by step and
write logits.

    bin/trace_run --model DIR --dtype bfloat16|float32 --out DIR --max-tokens N

Steps come on standard input, one JSON object a line:

    {"step": 0, "entries": [{"id": "a", "tokens": [5, 17], "want": [1]}],
     "end": ["a"]}

A step is one batch: each entry brings a request's next tokens and the places
among them whose logits are wanted; ``end`` lists requests that are finished
after it. The wanted logits go to DIR/<step>.f32, float32 [rows, vocab] in the
order of entries and places; ``done <step>`` on standard output follows every
step. The page pool holds --max-tokens tokens and there are state slots for
--max-requests live requests.

The engine runs the steps (LlmEngine.feed) with the batch, caches, kernels and
decode graphs that generation uses; nothing is sampled.
"""

import argparse
import json
import os
import sys
from typing import Dict


def _parse(argv):
    ap = argparse.ArgumentParser(prog="trace_run", description=(
        "Replay given tokens through a model and write logits."))
    ap.add_argument("--model", required=True,
                    help="folder with config.json and model.safetensors")
    ap.add_argument("--dtype", default="bfloat16",
                    choices=("bfloat16", "float32"))
    ap.add_argument("--out", required=True, help="folder for <step>.f32")
    ap.add_argument("--max-tokens", type=int, required=True,
                    help="most tokens that live requests hold at any time")
    ap.add_argument("--max-requests", type=int, default=4,
                    help="most live requests")
    ap.add_argument("--device", default=None,
                    help="cuda:N; cpu runs the reference operations")
    return ap.parse_args(argv)


def make_engine(args):
    from .engine import LlmEngine, LlmEngineConfig

    cfg = LlmEngineConfig.from_aux(args.model, {})
    if cfg.model_config is None:
        raise ValueError("no model family of this framework reads {}".format(
            os.path.join(args.model, "config.json")))
    cfg.dtype = args.dtype
    cfg.device = args.device
    cfg.max_num_seqs = args.max_requests
    cfg.num_kv_blocks = -(-args.max_tokens // cfg.block_size)
    cfg.max_model_len = cfg.num_kv_blocks * cfg.block_size
    engine = LlmEngine(cfg)
    engine.start()
    return engine


def run(engine, lines, out_dir: str, done) -> None:
    from .engine import SamplingParams, Sequence

    live: Dict[str, Sequence] = {}
    for line in lines:
        if not line.strip():
            continue
        step = json.loads(line)
        entries = []
        for e in step["entries"]:
            seq = live.get(e["id"])
            if seq is None:
                seq = live[e["id"]] = Sequence(e["id"], [], SamplingParams())
                engine.open_sequence(seq)
            if e["tokens"]:
                entries.append((seq, e["tokens"], e["want"]))
        if entries:
            # the copy to host memory also ends the step on the device
            logits = engine.feed(entries).float().cpu().numpy()
            if len(logits):
                path = os.path.join(out_dir, "{}.f32".format(step["step"]))
                logits.astype("<f4").tofile(path)
        for rid in step.get("end", []):
            engine.close_sequence(live.pop(rid))
        done(step["step"])


def main(argv=None) -> int:
    args = _parse(argv)
    if args.device != "cpu":
        from ...ops import reload_extensions
        from ...ops.build import ensure_library

        ensure_library("_hip_lm")
        reload_extensions()
        import torch

        if not torch.cuda.is_available():
            raise RuntimeError("no GPU found")
    engine = make_engine(args)

    def done(step):
        print("done {}".format(step), flush=True)

    run(engine, sys.stdin, args.out, done)
    return 0
