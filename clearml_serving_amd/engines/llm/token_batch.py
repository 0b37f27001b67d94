"""One forward's tokens: prompt portions and single tokens of different
sequences, flattened into one batch with no padding.

Entries are ordered by length, so that single tokens come first: kernels that
treat them apart (a recurrence step, absorbed attention) take a prefix of the
rows. All index arrays travel to the device in one copy.
"""

from typing import Any, Dict, List, Optional, Sequence as Seq

import numpy as np
import torch

from ...ops.grouped import pooled_row, token_row
from ...ops.lm import PROMPT_TILE


class TokenBatch:
    """Device-side description of a flat token batch.

    positions, slot_mapping, tok_seq [T]: position in the sequence, cache row
    (page * block_size + offset, -1: none), row of block_table;
    block_table [B, max pages]; state_slots [B];
    n_single: leading entries of one token (token i is entry i);
    n_abs: leading tokens whose attention runs in absorbed form;
    tiles [n, 5], seqs [m, 6]: recurrence tiles of the other entries (see
    ops.lm.rglru_prefill); prompts: per view -- a window, (window, first
    tokens that are kept) or (window, 0, tokens of a pooled block) -- the cache
    rows that the entries behind the first n_abs tokens can see and query tiles
    into them (see ops.lm.latent_prompt, ops.grouped.prompt); max_keys: bound on position + 1 in the first n_abs
    tokens."""

    mode = "token_batch"

    def __init__(self, **kw):
        self.__dict__.update(kw)

    @classmethod
    def build(cls, plan: Dict[str, Any], block_size: int, device,
              tile: int, absorb_max: Optional[int], windows: Seq):
        """plan: per entry "tokens", "starts", "blocks", "state_slots",
        "want" (places among its tokens whose logits are asked for).
        -> (tokens [T] int64, batch, wanted rows int32 in plan order)"""
        n = len(plan["tokens"])
        lens = [len(t) for t in plan["tokens"]]
        order = sorted(range(n), key=lambda i: lens[i])
        first = {}
        pos, slot, seq, toks = [], [], [], []
        tiles: List[List[int]] = []
        seqs: List[List[int]] = []
        n_single = n_abs = max_keys = at = 0
        gathered = {w: [] for w in windows}
        qtiles: Dict[Any, List[List[int]]] = {w: [] for w in windows}
        n_rows = dict.fromkeys(windows, 0)
        mb = max(len(b) for b in plan["blocks"])
        btab = np.zeros((n, mb), dtype=np.int32)
        for row, i in enumerate(order):
            start, ln = plan["starts"][i], lens[i]
            blocks = np.asarray(plan["blocks"][i], dtype=np.int32)
            btab[row, :len(blocks)] = blocks
            p = np.arange(start, start + ln, dtype=np.int32)
            first[i] = at
            toks.append(np.asarray(plan["tokens"][i], dtype=np.int64))
            pos.append(p)
            slot.append(blocks[p // block_size] * block_size + p % block_size)
            seq.append(np.full(ln, row, dtype=np.int32))
            sslot = plan["state_slots"][i]
            if ln == 1:
                n_single += 1
            else:
                t0 = len(tiles)
                for j in range(0, ln, tile):
                    tiles.append([at + j, min(tile, ln - j), start + j,
                                  sslot, j])
                seqs.append([t0, len(tiles) - t0, at, ln, start, sslot])
            at += ln
            if absorb_max is None or ln <= absorb_max:
                n_abs = at
                max_keys = max(max_keys, start + ln)
                continue
            for w in windows:
                size, keep, pool = (*w, 0)[:3] if isinstance(w, tuple) \
                    else (w, 0, 0)
                lo = max(0, start - size + 1) if size else 0
                keep = min(keep, lo)
                p = np.concatenate([
                    np.arange(keep, dtype=np.int32),
                    np.arange(lo, start + ln, dtype=np.int32)])
                rows = token_row(blocks[p // block_size], p % block_size,
                                 block_size, pool)
                n_pooled = []
                if pool:  # of the blocks that the last token sees
                    last = np.arange(pool - 1, start + ln - size, pool,
                                     dtype=np.int32)
                    rows = np.concatenate([
                        pooled_row(blocks[last // block_size],
                                   last % block_size, block_size, pool),
                        rows])
                    keep = len(last)
                    n_pooled = [keep]
                gathered[w].append(rows)
                for j in range(0, ln, PROMPT_TILE):
                    qtiles[w].append([first[i] + j, min(PROMPT_TILE, ln - j),
                                      start + j, n_rows[w], lo - keep,
                                      len(rows)] + n_pooled)
                n_rows[w] += len(rows)
        want = [first[i] + w for i in range(n) for w in plan["want"][i]]
        parts = {
            "positions": np.concatenate(pos),
            "slot_mapping": np.concatenate(slot),
            "tok_seq": np.concatenate(seq),
            "block_table": btab,
            "state_slots": np.asarray(
                [plan["state_slots"][i] for i in order], dtype=np.int32),
            "tiles": np.asarray(tiles, dtype=np.int32).reshape(-1, 5),
            "seqs": np.asarray(seqs, dtype=np.int32).reshape(-1, 6),
            "want": np.asarray(want, dtype=np.int32),
        }
        for w in windows:
            if qtiles[w]:
                parts["rows", w] = np.concatenate(gathered[w])
                # long-sighted tiles first
                parts["qtiles", w] = np.asarray(
                    sorted(qtiles[w], key=lambda q: -q[2]), dtype=np.int32)
        dev = to_device(parts, device)
        rows = dev.pop("want")
        prompts = {w: (dev.pop(("rows", w)), dev.pop(("qtiles", w)))
                   for w in windows if qtiles[w]}
        tokens = torch.from_numpy(np.concatenate(toks)).to(device)
        return tokens, cls(n_single=n_single, n_abs=n_abs, tile=tile,
                           max_keys=max_keys, prompts=prompts, **dev), rows

    @classmethod
    def of_single_tokens(cls, positions, slot_mapping, tok_seq, block_table,
                         state_slots, tile: int, max_keys: int):
        """n sequences, one token each, on given (static) tensors"""
        n = positions.shape[0]
        empty = torch.empty(0, dtype=torch.int32, device=positions.device)
        return cls(positions=positions, slot_mapping=slot_mapping,
                   tok_seq=tok_seq, block_table=block_table,
                   state_slots=state_slots, tiles=empty.view(0, 5),
                   seqs=empty.view(0, 6), n_single=n, n_abs=n, tile=tile,
                   max_keys=max_keys, prompts={})


def to_device(parts: Dict[str, np.ndarray], device) -> Dict[str, torch.Tensor]:
    """int32 arrays -> device tensors, one copy for all"""
    flat = np.concatenate([a.ravel() for a in parts.values()])
    dev = torch.from_numpy(flat).to(device)
    out, at = {}, 0
    for k, a in parts.items():
        out[k] = dev[at:at + a.size].view(a.shape)
        at += a.size
    return out
