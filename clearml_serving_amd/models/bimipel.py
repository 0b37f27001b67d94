"""Bimipel: a decoder of sliding-window latent attention and gated linear
recurrence layers, normalised on the sublayers' outputs.

    x = embed[token]
    x <- x + norm1(mixer(x));  x <- x + norm2(ff(x))   (ff where it has one)
    logits = logit_scale * embed @ norm(x)

The residual stream is float and is what the sublayers read; the norms'
weights are stored around zero. Layers are listed one by one in the
configuration, so order, sizes and windows are per layer. An attention layer
may use an earlier layer's cached latent instead of its own (``kv_from``).

Runs on flat token batches (engines/llm/token_batch.py): prompt portions and
single tokens of different sequences in one forward.
"""

import copy
from typing import Any, Dict, List, Optional

import torch
import torch.nn as nn

from ..ops import lm
from ..ops.lm import pad32
from . import register_arch, register_token_batch_arch
from .mixers import GatedMlp, LatentAttention, RgLru, _param, linear
from .token_lm import TokenBatchForCausalLM, TokenBatchLayer, held


class BimipelConfig:
    """``layers``: list of {"type", "mixer", "mlp"} as in config.json."""

    def __init__(self, raw: Dict[str, Any]):
        self.raw = copy.deepcopy(raw)
        self.vocab_size = int(raw["vocab"])
        self.hidden = int(raw["width"])
        self.eps = float(raw["norm"]["eps"])
        self.logit_scale = float(raw["logit_scale"])
        self.layers = self.raw["layers"]
        for n, layer in enumerate(self.layers):
            src = layer["mixer"].get("kv_from")
            if src is None:
                continue
            other = self.layers[src] if 0 <= src < n else None
            if (other is None or other["type"] != "latent_attention"
                    or other["mixer"].get("kv_from") is not None):
                raise ValueError(
                    "layer {}: kv_from {} is not an earlier attention layer "
                    "with a latent of its own".format(n, src))
            for key in ("kv_rank", "rot_dim", "rot"):
                if layer["mixer"][key] != other["mixer"][key]:
                    raise ValueError(
                        "layer {}: {} differs from layer {}, whose latent it "
                        "uses".format(n, key, src))


class BimipelLayer(TokenBatchLayer):
    def __init__(self, cfg: BimipelConfig, index: int):
        super().__init__()
        spec = cfg.layers[index]
        m = spec["mixer"]
        self.width, self.eps = cfg.hidden, cfg.eps
        if spec["type"] == "latent_attention":
            self.kv_from = m.get("kv_from")
            self.mix = LatentAttention(
                cfg.hidden, int(m["heads"]), int(m["dim"]),
                int(m["rot_dim"]), int(m["vdim"]), int(m["kv_rank"]),
                float(m["scale"]), int(m["mask"]["size"]),
                float(m["rot"]["base"]), int(m["rot"]["dims"]), cfg.eps,
                owns_kv=self.kv_from is None)
        elif spec["type"] == "rglru":
            self.kv_from = None
            self.mix = RgLru(cfg.hidden, int(m["width"]), int(m["blocks"]),
                             int(m["conv"]))
        else:
            raise ValueError("layer {}: unknown mixer '{}'".format(
                index, spec["type"]))
        wp = pad32(cfg.hidden)
        self.norm1 = _param(wp)
        self.mlp: Optional[GatedMlp] = None
        mlp = spec.get("mlp")
        if mlp is not None:
            if mlp["kind"] != "dense":
                raise ValueError("layer {}: unknown mlp kind '{}'".format(
                    index, mlp["kind"]))
            self.mlp = GatedMlp(cfg.hidden, int(mlp["ff"]))
            self.norm2 = _param(wp)

    def held(self):
        out = {"norm1": held(self.norm1, self.width)}
        if self.mlp is not None:
            out["norm2"] = held(self.norm2, self.width)
        return out

    def forward(self, x, h, batch, cache):
        h = lm.post_norm_add(self.mix(h, batch, cache), None, self.norm1, x,
                             self.width, self.eps)
        if self.mlp is not None:
            h = lm.post_norm_add(self.mlp(h), self.mlp.down_b, self.norm2, x,
                                 self.width, self.eps)
        return h


class BimipelForCausalLM(TokenBatchForCausalLM):
    def __init__(self, cfg: BimipelConfig):
        super().__init__()
        self.cfg = cfg
        wp = pad32(cfg.hidden)
        self.embed = _param(pad32(cfg.vocab_size), wp)
        self.layers = nn.ModuleList(
            [BimipelLayer(cfg, i) for i in range(len(cfg.layers))])
        self.final_norm = _param(wp)

    def held(self):
        c = self.cfg
        return {"embed": held(self.embed, c.vocab_size, c.hidden),
                "final.norm": held(self.final_norm, c.hidden)}

    def random_tensor(self, name, shape, gen):
        w = torch.empty(shape, dtype=torch.float32)
        if name.endswith("lam"):
            return w.uniform_(-4.0, 1.0, generator=gen)
        if name.endswith("dkv.norm"):
            return w.fill_(1.0)
        if len(shape) == 1:
            return w.normal_(std=0.02, generator=gen)
        return w.normal_(std=shape[-1] ** -0.5, generator=gen)

    def cache_layout(self) -> List[tuple]:
        out: List[tuple] = []
        for layer in self.layers:
            if isinstance(layer.mix, RgLru):
                wp, taps = layer.mix.wp, layer.mix.taps
                out.append(("state", (wp,), (taps, wp)))
            elif layer.kv_from is not None:
                out.append(("shared", layer.kv_from))
            else:
                out.append(("paged", layer.mix.row))
        return out

    # ---- forward ---------------------------------------------------- #
    def forward(self, tokens, positions, kv_caches, attn_ctx,
                last_token_idx=None, return_hidden=False,
                gather_logits=True):
        """attn_ctx: TokenBatch; logits [rows, vocab] at last_token_idx
        (int32; None: every token)"""
        x, h = lm.embed_stream(tokens, self.embed)
        for layer, cache in zip(self.layers, kv_caches):
            h = layer(x, h, attn_ctx, cache)
        c = self.cfg
        out = lm.output_norm(x, last_token_idx, self.final_norm, c.hidden,
                             c.eps, 1.0 if return_hidden else c.logit_scale)
        if return_hidden:
            return out[:, :c.hidden]
        logits = linear(out, self.embed)
        if logits.shape[1] != c.vocab_size:
            logits = logits[:, :c.vocab_size].contiguous()
        return logits


def _attn(heads, dim, rot, vdim, rank, window, base=10000.0, kv_from=None):
    m = {"heads": heads, "dim": dim, "rot_dim": rot, "vdim": vdim,
         "kv_rank": rank, "scale": (dim + rot) ** -0.5,
         "mask": {"size": window}, "rot": {"base": base, "dims": rot}}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return m


def _stack(vocab, width, ff, mixers) -> Dict[str, Any]:
    return {"architecture": "Bimipel", "vocab": vocab, "width": width,
            "norm": {"eps": 1e-6}, "logit_scale": 1.0,
            "layers": [{"type": t, "mixer": m,
                        "mlp": None if t == "rglru" and not f else
                        {"kind": "dense", "ff": ff}}
                       for t, m, f in mixers]}


def _griffin_like(vocab, width, ff, heads, dim, rot, rank, channels, blocks,
                  window, periods) -> Dict[str, Any]:
    rec = {"width": channels, "blocks": blocks, "conv": 4}
    mixers: List[tuple] = []
    for p in range(periods):
        src = len(mixers) - 3 if p % 2 else None  # every other pair shares
        mixers.append(("latent_attention",
                       _attn(heads, dim, rot, dim, rank, window,
                             kv_from=src), True))
        mixers.append(("rglru", dict(rec), True))
        mixers.append(("rglru", dict(rec), True))
    return _stack(vocab, width, ff, mixers)


PRESETS = {
    "bimipel-tiny": _stack(512, 96, 160, [
        ("latent_attention", _attn(3, 32, 16, 24, 40, 24), True),
        ("rglru", {"width": 144, "blocks": 3, "conv": 3}, False),
        ("latent_attention", _attn(2, 24, 16, 40, 40, 9, kv_from=0), True),
    ]),
    # llama-3-1b's width, depth class and vocabulary
    "bimipel-1b": _griffin_like(128256, 2048, 6144, 16, 96, 32, 384, 2560,
                                20, 1024, 6),
    "bimipel-300m": _griffin_like(32000, 1024, 3072, 8, 96, 32, 256, 1280,
                                  10, 512, 4),
    # six layers as wide as an 8B model's
    "bimipel-4k": _griffin_like(32000, 4096, 12288, 32, 96, 32, 512, 4096,
                                16, 2048, 2),
}


def _build(config: Optional[Dict[str, Any]] = None,
           preset: str = "bimipel-tiny",
           overrides: Optional[Dict[str, Any]] = None) -> BimipelForCausalLM:
    raw = dict(config if config is not None else PRESETS[preset])
    raw.update(overrides or {})
    return BimipelForCausalLM(BimipelConfig(raw))


register_token_batch_arch("bimipel", _build, architecture="Bimipel")


@register_arch("bimipel")
def bimipel(preset: str = "bimipel-tiny", config=None,
            **overrides) -> BimipelForCausalLM:
    return _build(config, preset, overrides)
