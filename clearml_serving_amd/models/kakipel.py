"""Kakipel: a decoder of latent attention layers with gated outputs and
queries from a latent of their own, norms before and after every sublayer,
dense or mixture-of-experts feed-forwards, and a stretch of layers that runs
several times.

    x = x0 = embed[token]
    before each pass of the loop:  x <- W_in [x; x0] + step[pass]
    x <- x + norm1b(mixer(norm1(x)));  x <- x + norm2b(ff(norm2(x)))
    logits = head norm(x)

The residual stream x is float; every kernel that changes it also writes the
norm (or, in front of a pass, the copy) that the next product reads. The loop's
passes share weights and have a cache each, so the engine sees one cache per
layer *run*.

Runs on flat token batches (engines/llm/token_batch.py): prompt portions and
single tokens of different sequences in one forward.
"""

import copy
from typing import Any, Dict, List, Optional, Tuple

import torch
import torch.nn as nn

from ..ops import lm
from ..ops.lm import RowNorm, pad32
from . import register_arch, register_token_batch_arch
from .mixers import ExpertMlp, GatedMlp, LatentAttention, _param, linear
from .token_lm import TokenBatchForCausalLM, TokenBatchLayer, held


class KakipelConfig:
    """``layers``: list of {"type", "mixer", "mlp"}; ``loop``: start, stop,
    times or absent, as in config.json."""

    def __init__(self, raw: Dict[str, Any]):
        self.raw = copy.deepcopy(raw)
        self.vocab_size = int(raw["vocab"])
        self.hidden = int(raw["width"])
        self.eps = float(raw["norm"]["eps"])
        self.layers = self.raw["layers"]
        n, loop = len(self.layers), raw.get("loop")
        self.loop: Optional[Tuple[int, int, int]] = None
        # layer runs in order: (layer, pass that begins right before it)
        self.runs: List[Tuple[int, Optional[int]]] = [(i, None)
                                                      for i in range(n)]
        if loop is not None:
            start, stop, times = (int(loop[k])
                                  for k in ("start", "stop", "times"))
            if not (0 <= start < stop <= n and times >= 1):
                raise ValueError("loop {} does not fit {} layers".format(
                    loop, n))
            self.loop = start, stop, times
            self.runs[start:stop] = [
                (i, t if i == start else None)
                for t in range(times) for i in range(start, stop)]


def _feed_forward(cfg: KakipelConfig, index: int, mlp: Dict[str, Any]):
    if mlp["kind"] == "dense":
        return GatedMlp(cfg.hidden, int(mlp["ff"]), act="silu", bias=False)
    if mlp["kind"] == "moe":
        return ExpertMlp(cfg.hidden, int(mlp["expert"]["ff"]),
                         int(mlp["router"]["experts"]),
                         int(mlp["router"]["top"]), act="relu2")
    raise ValueError("layer {}: unknown mlp kind '{}'".format(
        index, mlp["kind"]))


class KakipelLayer(TokenBatchLayer):
    def __init__(self, cfg: KakipelConfig, index: int):
        super().__init__()
        spec = cfg.layers[index]
        if spec["type"] != "latent_attention":
            raise ValueError("layer {}: unknown mixer '{}'".format(
                index, spec["type"]))
        m, rot = spec["mixer"], spec["mixer"]["rot"]
        self.width, self.eps = cfg.hidden, cfg.eps
        self.mix = LatentAttention(
            cfg.hidden, int(m["heads"]), int(m["dim"]), int(m["rot_dim"]),
            int(m["vdim"]), int(m["kv_rank"]), float(m["scale"]), 0,
            float(rot["base"]), int(rot["dims"]), cfg.eps,
            q_rank=int(m["q_rank"]), rot_half=True,
            rot_scaling=rot.get("scaling"), sink=False, gate=True)
        wp = pad32(cfg.hidden)
        self.norm1, self.norm1b = _param(wp), _param(wp)
        mlp = spec.get("mlp")
        self.mlp = None if mlp is None else _feed_forward(cfg, index, mlp)
        if mlp is not None:
            self.norm2, self.norm2b = _param(wp), _param(wp)

    def held(self):
        names = ["norm1", "norm1b"]
        if self.mlp is not None:
            names += ["norm2", "norm2b"]
        return {k: held(getattr(self, k), self.width) for k in names}

    def norm_in(self) -> RowNorm:
        return RowNorm(self.norm1, self.width, self.eps, 0.0)

    def forward(self, x, h, batch, cache, norm, out=None):
        """h: norm1(x). Returns norm(x) of the new x (x itself without a
        norm), in ``out`` if given."""
        def add(o, weight, norm, out=None, mix=None):
            return lm.post_norm_add(o, None, weight, x, self.width, self.eps,
                                    0.0, norm, out, mix)

        o = self.mix(h, batch, cache)
        if self.mlp is None:
            return add(o, self.norm1b, norm, out)
        h = add(o, self.norm1b,
                RowNorm(self.norm2, self.width, self.eps, 0.0))
        if isinstance(self.mlp, ExpertMlp):
            o, mix = self.mlp(h)
            return add(o, self.norm2b, norm, out, mix)
        return add(self.mlp(h), self.norm2b, norm, out)


class KakipelForCausalLM(TokenBatchForCausalLM):
    def __init__(self, cfg: KakipelConfig):
        super().__init__()
        self.cfg = cfg
        wp, vp = pad32(cfg.hidden), pad32(cfg.vocab_size)
        self.wp = wp
        self.embed = _param(vp, wp)
        self.head = _param(vp, wp)
        self.final_norm = _param(wp)
        self.layers = nn.ModuleList(
            [KakipelLayer(cfg, i) for i in range(len(cfg.layers))])
        if cfg.loop is not None:
            self.loop_in = _param(wp, 2, wp)  # columns [x | x0]
            self.loop_step = _param(cfg.loop[2], wp)

    def held(self):
        c = self.cfg
        v, w = c.vocab_size, c.hidden
        out = {"embed": held(self.embed, v, w), "head": held(self.head, v, w),
               "final.norm": held(self.final_norm, w)}
        if c.loop is not None:
            out["loop.in"] = held(self.loop_in, w, 2 * w, fill_as=(w, 2, w))
            out["loop.step"] = held(self.loop_step, c.loop[2], w)
        return out

    def ignored(self):
        return ["l{}.{}".format(i, k) for i, m in enumerate(self.layers)
                if m.mlp is None for k in ("norm2", "norm2b")]

    def random_tensor(self, name, shape, gen):
        w = torch.empty(shape, dtype=torch.float32)
        if name == "loop.step":
            return w.normal_(std=0.02, generator=gen)
        if len(shape) == 1:  # norms
            return w.normal_(mean=1.0, std=0.02, generator=gen)
        return w.normal_(std=shape[-1] ** -0.5, generator=gen)

    def cache_layout(self) -> List[tuple]:
        return [("paged", self.layers[i].mix.row) for i, _ in self.cfg.runs]

    # ---- forward ---------------------------------------------------- #
    def forward(self, tokens, positions, kv_caches, attn_ctx,
                last_token_idx=None, return_hidden=False,
                gather_logits=True):
        """attn_ctx: TokenBatch; logits [rows, vocab] at last_token_idx
        (int32; None: every token)"""
        c, wp = self.cfg, self.wp
        entry = left = right = None
        if c.loop is not None:  # what enters a pass: [x | x0]
            entry = self.embed.new_empty(tokens.shape[0], 2 * wp)
            left, right = entry[:, :wp], entry[:, wp:]
        # per run, what the kernel in front of it writes
        before = [(None, left) if t is not None else
                  (self.layers[i].norm_in(), None) for i, t in c.runs]
        before.append((RowNorm(self.final_norm, c.hidden, c.eps, 0.0), None))
        norm, out = before[0]
        x, h = lm.embed_stream(tokens, self.embed, norm, out, right)
        for r, (i, t) in enumerate(c.runs):
            layer = self.layers[i]
            if t is not None:
                x = lm.linear_f32(entry, self.loop_in.view(wp, 2 * wp))
                h = lm.add_norm(x, self.loop_step[t], layer.norm_in())
            h = layer(x, h, attn_ctx, kv_caches[r], *before[r + 1])
        if last_token_idx is not None:
            h = lm.gather_rows(h, last_token_idx)
        if return_hidden:
            return h[:, :c.hidden]
        logits = linear(h, self.head)
        if logits.shape[1] != c.vocab_size:
            logits = logits[:, :c.vocab_size].contiguous()
        return logits


def _attn(heads, dim, rot, vdim, q_rank, rank, base=10000.0, factor=8.0,
          original=4096):
    return {"heads": heads, "dim": dim, "rot_dim": rot, "vdim": vdim,
            "q_rank": q_rank, "kv_rank": rank, "scale": (dim + rot) ** -0.5,
            "rot": {"base": base, "dims": rot, "scaling": {
                "factor": factor, "original": original, "fast": 32.0,
                "slow": 1.0}}}


def _stack(vocab, width, mixer, n, ff, expert_ff, experts, top, loop
           ) -> Dict[str, Any]:
    """n layers, every second one a mixture of experts"""
    moe = {"kind": "moe", "expert": {"ff": expert_ff},
           "router": {"experts": experts, "top": top}}
    start, stop, times = loop
    return {"architecture": "Kakipel", "vocab": vocab, "width": width,
            "norm": {"eps": 1e-6},
            "loop": {"start": start, "stop": stop, "times": times},
            "layers": [{"type": "latent_attention", "mixer": dict(mixer),
                        "mlp": moe if i % 2 else {"kind": "dense", "ff": ff}}
                       for i in range(n)]}


PRESETS = {
    "kakipel-tiny": _stack(512, 96, _attn(3, 24, 16, 40, 56, 48), 3, 160, 48,
                           6, 2, (1, 3, 2)),
    "kakipel-300m": _stack(32000, 1024, _attn(8, 96, 32, 96, 512, 256), 8,
                           3072, 768, 16, 4, (2, 4, 3)),
    # llama-3-1b's width and vocabulary
    "kakipel-1b": _stack(128256, 2048, _attn(16, 96, 32, 96, 768, 384), 8,
                         6144, 1536, 16, 4, (2, 4, 3)),
    # layers as wide as an 8B model's
    "kakipel-4k": _stack(32000, 4096, _attn(32, 96, 32, 96, 1536, 512), 4,
                         12288, 2560, 16, 4, (0, 2, 2)),
}


def _build(config: Optional[Dict[str, Any]] = None,
           preset: str = "kakipel-tiny",
           overrides: Optional[Dict[str, Any]] = None) -> KakipelForCausalLM:
    raw = dict(config if config is not None else PRESETS[preset])
    raw.update(overrides or {})
    return KakipelForCausalLM(KakipelConfig(raw))


register_token_batch_arch("kakipel", _build, architecture="Kakipel")


@register_arch("kakipel")
def kakipel(preset: str = "kakipel-tiny", config=None,
            **overrides) -> KakipelForCausalLM:
    return _build(config, preset, overrides)
