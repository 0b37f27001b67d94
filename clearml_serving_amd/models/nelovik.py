"""Nelovik: a decoder whose mixer and feed-forward stand side by side in every
layer, with gated delta rules, and layers of windowed attention over pooled
history beside a state-space recurrence.

    x = embed[token]
    per layer:  x <- x + mixer(norm1(x)) + mlp(norm2(x))
    logits = head norm(x)

The stream is float. Both norms of a layer share their root mean square: the
kernel that adds a layer's outputs to the stream also writes the two inputs of
the next one. A recurrent mixer and the feed-forward have one output product.

Runs on flat token batches (engines/llm/token_batch.py): prompt portions and
single tokens of different sequences in one forward.
"""

import copy
from typing import Any, Dict, List, Optional

import torch
import torch.nn as nn

from ..ops import lm
from ..ops.lm import RowNorm, pad32
from . import register_arch, register_token_batch_arch
from .mixers import (DenseMlp, GatedDelta, GroupedAttention, ParallelMixer,
                     RecurrentMixer, StateSpace, _param, linear)
from .token_lm import TokenBatchForCausalLM, TokenBatchLayer, held


class NelovikConfig:
    """``layers``: list of {"type", "mixer", "mlp"} as in config.json."""

    def __init__(self, raw: Dict[str, Any]):
        self.raw = copy.deepcopy(raw)
        self.vocab_size = int(raw["vocab"])
        self.hidden = int(raw["width"])
        self.eps = float(raw["norm"]["eps"])
        self.layers = self.raw["layers"]


def _delta(cfg: NelovikConfig, m: Dict[str, Any]) -> nn.Module:
    return RecurrentMixer(cfg.hidden, GatedDelta(
        cfg.hidden, int(m["heads"]), int(m["kv_heads"]), int(m["dim"]),
        int(m["vdim"]), int(m["conv"]), cfg.eps))


def _parallel(cfg: NelovikConfig, m: Dict[str, Any]) -> nn.Module:
    a, s = m["left"], m["right"]
    rot, mask = a["rot"], a["mask"]
    left = GroupedAttention(
        cfg.hidden, int(a["heads"]), int(a["kv_heads"]), int(a["dim"]),
        int(a["vdim"]), float(a["scale"]), cfg.eps,
        rot=(float(rot["base"]), int(rot["dims"]), 1.0), rot_half=True,
        window=int(mask["size"]), pool=int(mask["pool"]),
        cap=float(a["softcap"]), qk_norm="all", sink="learned", bias=True)
    right = StateSpace(
        cfg.hidden, int(s["heads"]), int(s["vdim"]), int(s["state"]),
        int(s["groups"]), int(s["conv"]), int(s["norm_groups"]), cfg.eps)
    return ParallelMixer(cfg.hidden, left, 0.5, right, 0.5, norm_outputs=True)


MIXERS = {"parallel": _parallel, "delta": _delta, "delta_2": _delta}


class NelovikLayer(TokenBatchLayer):
    def __init__(self, cfg: NelovikConfig, index: int):
        super().__init__()
        spec = cfg.layers[index]
        if spec["type"] not in MIXERS:
            raise ValueError("layer {}: unknown mixer '{}'".format(
                index, spec["type"]))
        self.width, self.eps = cfg.hidden, cfg.eps
        self.mix = MIXERS[spec["type"]](cfg, spec["mixer"])
        self.mlp, mlp, wp = None, spec.get("mlp"), pad32(cfg.hidden)
        if mlp is not None:
            if mlp["kind"] != "dense":
                raise ValueError("layer {}: unknown mlp kind '{}'".format(
                    index, mlp["kind"]))
            self.mlp = DenseMlp(cfg.hidden, int(mlp["ff"]))
        self.norm1 = _param(wp)
        self.norm2 = None if mlp is None else _param(wp)
        # columns of the output product: the mixer's, unless it has its own,
        # and the feed-forward's
        self.merged = isinstance(self.mix, RecurrentMixer)
        self.cut = self.mix.out_cols if self.merged else 0
        cols = self.cut + (0 if mlp is None else self.mlp.out_cols)
        self.o = _param(wp, cols) if cols else None

    def held(self):
        out = {"norm1": held(self.norm1, self.width)}
        if self.norm2 is not None:
            out["norm2"] = held(self.norm2, self.width)
        return out

    def pack_shared(self, get) -> None:
        if self.merged:
            self.mix.pack_out(self.o.data[:, :self.cut],
                              lambda name: get("mix." + name))
        if self.mlp is not None:
            self.mlp.pack_out(self.o.data[:, self.cut:],
                              lambda name: get("mlp." + name))

    def norms_in(self) -> List[RowNorm]:
        return [RowNorm(w.data, self.width, self.eps, 0.0)
                for w in (self.norm1, self.norm2) if w is not None]

    def forward(self, x, h, batch, cache, norms):
        """h: the inputs of mixer and feed-forward. -> norm(x) of the new x
        for each of ``norms``"""
        plain, branches = None, []
        if self.o is not None:
            ctx = h[0].new_empty(x.shape[0], self.o.shape[1])
        if self.merged:
            self.mix.context(h[0], batch, cache, ctx[:, :self.cut])
        else:
            branches = self.mix.branches(h[0], batch, cache)
        if self.mlp is not None:
            self.mlp.context(h[1], ctx[:, self.cut:])
        if self.o is not None:
            plain = linear(ctx, self.o)
        return lm.add_branches(
            x, plain, branches, 0.0 if self.merged else self.mix.scale,
            norms, self.width, self.eps, self.norm1.dtype)


class NelovikForCausalLM(TokenBatchForCausalLM):
    def __init__(self, cfg: NelovikConfig):
        super().__init__()
        self.cfg = cfg
        wp, vp = pad32(cfg.hidden), pad32(cfg.vocab_size)
        self.embed = _param(vp, wp)
        self.head = _param(vp, wp)
        self.final_norm = _param(wp)
        self.layers = nn.ModuleList(
            [NelovikLayer(cfg, i) for i in range(len(cfg.layers))])

    def held(self):
        v, w = self.cfg.vocab_size, self.cfg.hidden
        return {"embed": held(self.embed, v, w), "head": held(self.head, v, w),
                "final.norm": held(self.final_norm, w)}

    def ignored(self):
        return ["l{}.norm2".format(i) for i, m in enumerate(self.layers)
                if m.mlp is None]

    def random_tensor(self, name, shape, gen):
        w = torch.empty(shape, dtype=torch.float32)
        leaf = name.split(".")[-1]
        if leaf in ("norm", "norm1", "norm2", "out", "D"):
            return w.normal_(mean=1.0, std=0.02, generator=gen)
        if leaf == "A_log":  # rates of 1 to 16
            return w.uniform_(1.0, 16.0, generator=gen).log_()
        if leaf == "dt_bias":  # steps of 0.001 to 0.1
            return torch.expm1(torch.exp(
                w.uniform_(-6.9, -2.3, generator=gen))).log_()
        if leaf == "act":
            return w.fill_(0.8)
        if len(shape) == 1:  # biases, sinks
            return w.normal_(std=0.02, generator=gen)
        return w.normal_(std=shape[-1] ** -0.5, generator=gen)

    def load_checkpoint(self, state: Dict[str, torch.Tensor]) -> None:
        super().load_checkpoint(state)
        for i, layer in enumerate(self.layers):
            layer.pack_shared(lambda name, q="l{}.".format(i):
                              state[q + name])

    def cache_layout(self) -> List[tuple]:
        return [layer.mix.cache_layout() for layer in self.layers]

    # ---- forward ---------------------------------------------------- #
    def forward(self, tokens, positions, kv_caches, attn_ctx,
                last_token_idx=None, return_hidden=False,
                gather_logits=True):
        """attn_ctx: TokenBatch; logits [rows, vocab] at last_token_idx
        (int32; None: every token)"""
        c = self.cfg
        final = RowNorm(self.final_norm.data, c.hidden, c.eps, 0.0)
        # of selected rows the output norm is a step of its own
        last = [final] if last_token_idx is None else []
        norms = [layer.norms_in() for layer in self.layers] + [last]
        if norms[0]:
            x, h = lm.embed_norms(tokens, self.embed, norms[0])
        else:  # no layers
            x, h = lm.embed_stream(tokens, self.embed)
        for layer, cache, nxt in zip(self.layers, kv_caches, norms[1:]):
            h = layer(x, h, attn_ctx, cache, nxt)
        if last:
            h = h[0]
        else:
            h = lm.output_norm(x, last_token_idx, self.final_norm, c.hidden,
                               c.eps, offset=0.0)
        if return_hidden:
            return h[:, :c.hidden]
        return linear(h, self.head)[:, :c.vocab_size]


def _delta_spec(heads, kv, dim, vdim, taps=4):
    return {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim,
            "conv": taps}


def _parallel_spec(heads, kv, dim, vdim, rot, window, pool, s_heads, s_vdim,
                   state, groups, parts):
    return {"left": {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim,
                     "scale": dim ** -0.5, "softcap": 50.0,
                     "rot": {"base": 10000.0, "dims": rot},
                     "mask": {"size": window, "pool": pool}},
            "right": {"heads": s_heads, "vdim": s_vdim, "state": state,
                      "groups": groups, "conv": 4, "norm_groups": parts}}


def _stack(vocab, width, ff, delta, par, n) -> Dict[str, Any]:
    """n layers, every third one of the parallel kind"""
    return {"architecture": "Nelovik", "vocab": vocab, "width": width,
            "norm": {"eps": 1e-6},
            "layers": [{"type": t, "mixer": copy.deepcopy(m),
                        "mlp": {"kind": "dense", "ff": ff}}
                       for t, m in (("parallel", par) if i % 3 == 2 else
                                    ("delta", delta) for i in range(n))]}


PRESETS = {
    "nelovik-tiny": _stack(
        512, 96, 160, _delta_spec(4, 2, 24, 40),
        _parallel_spec(4, 2, 24, 40, 12, 24, 6, 6, 16, 40, 2, 3), 3),
    "nelovik-300m": _stack(
        32000, 1024, 3584, _delta_spec(16, 8, 64, 64),
        _parallel_spec(16, 4, 64, 64, 32, 512, 16, 32, 64, 64, 2, 2), 12),
    # llama-3-1b's width and vocabulary
    "nelovik-1b": _stack(
        128256, 2048, 8192, _delta_spec(16, 16, 128, 128),
        _parallel_spec(32, 8, 64, 64, 32, 1024, 16, 64, 64, 128, 8, 8), 12),
    # layers as wide as an 8B model's
    "nelovik-4k": _stack(
        32000, 4096, 12288, _delta_spec(32, 16, 128, 128),
        _parallel_spec(32, 8, 128, 128, 64, 2048, 16, 128, 64, 128, 8, 8), 6),
}


def _build(config: Optional[Dict[str, Any]] = None,
           preset: str = "nelovik-tiny",
           overrides: Optional[Dict[str, Any]] = None) -> NelovikForCausalLM:
    raw = dict(config if config is not None else PRESETS[preset])
    raw.update(overrides or {})
    return NelovikForCausalLM(NelovikConfig(raw))


register_token_batch_arch("nelovik", _build, architecture="Nelovik")


@register_arch("nelovik")
def nelovik(preset: str = "nelovik-tiny", config=None,
            **overrides) -> NelovikForCausalLM:
    return _build(config, preset, overrides)
