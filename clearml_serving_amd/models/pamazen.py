"""Pamazen: a decoder on hyper-connected residual streams, with grouped-query
attention layers whose values mix with the first such layer's, layers of
windowed attention and a generalised delta rule side by side, and mixtures of
gated, shared and identity experts.

    X_1 .. X_S = embed[token]
    per sublayer:  u = sum_s in[s] X_s;  y = sublayer(norm(u))
                   X_t <- sum_s mix[s, t] X_s + m out[t] y
    logits = cap tanh(head norm(sum_s X_s) / cap)

The streams are float; the kernel that returns a sublayer's output to them also
writes the norm that the next sublayer reads. A norm's weight is one number.

Runs on flat token batches (engines/llm/token_batch.py): prompt portions and
single tokens of different sequences in one forward.
"""

import copy
from typing import Any, Dict, List, Optional

import torch
import torch.nn as nn

from ..ops import hyper, lm
from ..ops.lm import pad32
from . import register_arch, register_token_batch_arch
from .mixers import (DeltaRule, ExpertMlp, GroupedAttention,
                     GroupedAttentionMixer, ParallelMixer, _param, linear)
from .token_lm import TokenBatchForCausalLM, TokenBatchLayer, held


class PamazenConfig:
    """``layers``: list of {"type", "mixer", "mlp"} as in config.json."""

    def __init__(self, raw: Dict[str, Any]):
        self.raw = copy.deepcopy(raw)
        self.vocab_size = int(raw["vocab"])
        self.hidden = int(raw["width"])
        self.eps = float(raw["norm"]["eps"])
        self.streams = int(raw["streams"])
        self.residual_mult = float(raw["residual_mult"])
        self.logit_softcap = float(raw["logit_softcap"])
        self.layers = self.raw["layers"]
        if not 1 <= self.streams <= hyper.MAX_STREAMS:
            raise ValueError("{} residual streams, 1 to {} are possible"
                             .format(self.streams, hyper.MAX_STREAMS))
        sizes = {(lay["mixer"]["kv_heads"], lay["mixer"]["vdim"])
                 for lay in self.layers
                 if lay["type"] == "attention" and lay["mixer"].get("v_mix")}
        if len(sizes) > 1:
            raise ValueError("layers that mix their values have different "
                             "values: {}".format(sorted(sizes)))


def _attention(cfg: PamazenConfig, m: Dict[str, Any]) -> nn.Module:
    rot = m["rot"]
    factor = (rot.get("scaling") or {}).get("factor", 1.0)
    return GroupedAttentionMixer(
        cfg.hidden, int(m["heads"]), int(m["kv_heads"]), int(m["dim"]),
        int(m["vdim"]), float(m["scale"]),
        rot=(float(rot["base"]), int(rot["dims"]), float(factor)),
        sink="one", v_mix=bool(m.get("v_mix", False)))


def _parallel(cfg: PamazenConfig, m: Dict[str, Any]) -> nn.Module:
    a, d = m["left"], m["right"]
    left = GroupedAttention(
        cfg.hidden, int(a["heads"]), int(a["kv_heads"]), int(a["dim"]),
        int(a["vdim"]), float(a["scale"]), cfg.eps,
        window=int(a["mask"]["size"]),
        keep=int(a["mask"].get("keep_first", 0)), cap=float(a["softcap"]),
        qk_norm=True, values_are_keys=True, sink="learned")
    right = DeltaRule(cfg.hidden, int(d["heads"]), int(d["dim"]), cfg.eps)
    return ParallelMixer(cfg.hidden, left, float(m["left_scale"]), right,
                         float(m["right_scale"]))


MIXERS = {"attention": _attention, "parallel": _parallel}


def _feed_forward(cfg: PamazenConfig, index: int,
                  mlp: Dict[str, Any]) -> ExpertMlp:
    if mlp["kind"] != "moe":
        raise ValueError("layer {}: unknown mlp kind '{}'".format(
            index, mlp["kind"]))
    r, groups, shared = mlp["router"], mlp["router"].get("groups"), \
        mlp.get("shared")
    return ExpertMlp(
        cfg.hidden, int(mlp["expert"]["ff"]), int(r["experts"]),
        int(r["top"]), act="silu", gated=True, correction=True,
        groups=None if groups is None else (int(groups["count"]),
                                            int(groups["keep"])),
        identity=int(r.get("identity", 0)),
        shared_ff=None if shared is None else int(shared["ff"]))


class HyperConnection(nn.Module):
    """One sublayer's norm gain and weights of the streams."""

    def __init__(self, streams: int):
        super().__init__()
        self.w_in, self.w_out = _param(streams), _param(streams)
        self.mix = _param(streams, streams)
        self.gain = _param()


class PamazenLayer(TokenBatchLayer):
    def __init__(self, cfg: PamazenConfig, index: int):
        super().__init__()
        spec = cfg.layers[index]
        if spec["type"] not in MIXERS:
            raise ValueError("layer {}: unknown mixer '{}'".format(
                index, spec["type"]))
        self.width, self.eps, self.streams = cfg.hidden, cfg.eps, cfg.streams
        self.mix = MIXERS[spec["type"]](cfg, spec["mixer"])
        mlp = spec.get("mlp")
        self.mlp = None if mlp is None else _feed_forward(cfg, index, mlp)
        self.hc = nn.ModuleList([HyperConnection(cfg.streams) for _ in
                                 range(1 if mlp is None else 2)])
        # per sublayer, what its step needs (set by the model's finalize)
        self.coef: List[torch.Tensor] = []
        self.last = False

    def held(self):
        s, out = self.streams, {}
        for q, hc in enumerate(self.hc, 1):
            out["norm{}".format(q)] = held(hc.gain)
            out["hc{}.in".format(q)] = held(hc.w_in, s)
            out["hc{}.out".format(q)] = held(hc.w_out, s)
            out["hc{}.mix".format(q)] = held(hc.mix, s, s)
        return out

    def forward(self, x, h, batch, cache, carry):
        """h: the first sublayer's normed input. Returns the next layer's."""
        n, eps = self.width, self.eps
        o = self.mix(h, batch, cache, carry)
        if self.mlp is None:
            return hyper.step(o, x, self.coef[0], n, eps, self.last)
        h = hyper.step(o, x, self.coef[0], n, eps)
        rows, mix = self.mlp(h)
        return hyper.step(rows, x, self.coef[1], n, eps, self.last, mix,
                          h if self.mlp.has_skip else None)


class PamazenForCausalLM(TokenBatchForCausalLM):
    def __init__(self, cfg: PamazenConfig):
        super().__init__()
        self.cfg = cfg
        wp, vp = pad32(cfg.hidden), pad32(cfg.vocab_size)
        self.embed = _param(vp, wp)
        self.head = _param(vp, wp)
        self.final_norm = _param()
        self.layers = nn.ModuleList(
            [PamazenLayer(cfg, i) for i in range(len(cfg.layers))])
        self.entry: Optional[torch.Tensor] = None

    def held(self):
        v, w = self.cfg.vocab_size, self.cfg.hidden
        return {"embed": held(self.embed, v, w), "head": held(self.head, v, w),
                "final.norm": held(self.final_norm)}

    def ignored(self):
        """of sublayers that are not there, and of layers that do not mix"""
        out = []
        for i, m in enumerate(self.layers):
            names = ["mix.vmix"]
            if m.mlp is None:
                names += ["norm2", "hc2.in", "hc2.out", "hc2.mix"]
            out += ["l{}.{}".format(i, k) for k in names]
        return out

    def random_tensor(self, name, shape, gen):
        w = torch.empty(shape, dtype=torch.float32)
        s, leaf = self.cfg.streams, name.split(".")[-1]
        if ".hc" in name:
            base = {"in": torch.full((s,), 1.0 / s), "out": torch.ones(s),
                    "mix": torch.eye(s)}[leaf]
            return base + w.normal_(std=0.02, generator=gen)
        if leaf == "vmix":
            return w.fill_(0.5)
        if leaf in ("norm", "norm1", "norm2"):
            return w.normal_(mean=1.0, std=0.02, generator=gen)
        if len(shape) == 1:  # sinks, corrections, decay and rate offsets
            return w.normal_(std=0.02, generator=gen)
        return w.normal_(std=shape[-1] ** -0.5, generator=gen)

    def finalize(self) -> None:
        super().finalize()
        hcs = [hc for layer in self.layers for hc in layer.hc]
        # what reads the streams behind each sublayer: the next one, and in
        # the end the output norm of their sum
        ends = torch.ones(self.cfg.streams, device=self.embed.device)
        reads = [(hc.w_in, hc.gain) for hc in hcs] + [(ends, self.final_norm)]
        self.entry = hyper.entry_coef(*reads[0])
        steps = [hyper.step_coef(hc.mix, hc.w_out, self.cfg.residual_mult,
                                 *nxt) for hc, nxt in zip(hcs, reads[1:])]
        for layer in self.layers:
            layer.coef = [steps.pop(0) for _ in layer.hc]
        if len(self.layers):
            self.layers[-1].last = True

    def cache_layout(self) -> List[tuple]:
        return [layer.mix.cache_layout() for layer in self.layers]

    # ---- forward ---------------------------------------------------- #
    def forward(self, tokens, positions, kv_caches, attn_ctx,
                last_token_idx=None, return_hidden=False,
                gather_logits=True):
        """attn_ctx: TokenBatch; float logits [rows, vocab] at last_token_idx
        (int32; None: every token)"""
        c = self.cfg
        x, h = hyper.embed(tokens, self.embed, self.entry, c.streams,
                           c.hidden, c.eps)
        carry: Dict[str, torch.Tensor] = {}
        for layer, cache in zip(self.layers, kv_caches):
            h = layer(x, h, attn_ctx, cache, carry)
        if last_token_idx is not None:
            h = lm.gather_rows(h, last_token_idx)
        if return_hidden:
            return h[:, :c.hidden]
        return hyper.soft_cap(linear(h, self.head), c.vocab_size,
                              c.logit_softcap)


def _moe(ff, experts, top, identity, groups, keep, shared):
    return {"kind": "moe", "expert": {"ff": ff}, "shared": {"ff": shared},
            "router": {"experts": experts, "top": top, "identity": identity,
                       "groups": {"count": groups, "keep": keep}}}


def _attn_spec(heads, kv, dim, rot, vdim, base=10000.0, factor=4.0):
    return {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim,
            "scale": dim ** -0.5, "v_mix": True,
            "rot": {"base": base, "dims": rot, "scaling": {"factor": factor}}}


def _parallel_spec(heads, kv, dim, window, keep, r_heads, r_dim):
    return {"left": {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": dim,
                     "scale": dim ** -0.5, "softcap": 30.0,
                     "mask": {"size": window, "keep_first": keep}},
            "right": {"heads": r_heads, "dim": r_dim},
            "left_scale": 1.0, "right_scale": 1.0}


def _stack(vocab, width, streams, attn, par, n, mlp) -> Dict[str, Any]:
    """n layers, every third one of the parallel kind"""
    return {"architecture": "Pamazen", "vocab": vocab, "width": width,
            "norm": {"eps": 1e-6}, "streams": streams, "residual_mult": 1.0,
            "logit_softcap": 30.0,
            "layers": [{"type": t, "mixer": copy.deepcopy(m),
                        "mlp": copy.deepcopy(mlp)}
                       for t, m in (("parallel", par) if i % 3 == 2 else
                                    ("attention", attn) for i in range(n))]}


PRESETS = {
    "pamazen-tiny": _stack(512, 96, 3, _attn_spec(4, 2, 24, 16, 40),
                           _parallel_spec(6, 2, 40, 24, 3, 2, 48), 3,
                           _moe(48, 6, 2, 2, 4, 3, 80)),
    "pamazen-300m": _stack(32000, 1024, 4, _attn_spec(16, 4, 64, 64, 64),
                           _parallel_spec(16, 4, 64, 512, 16, 16, 64), 9,
                           _moe(384, 12, 4, 4, 4, 3, 384)),
    # llama-3-1b's width and vocabulary
    "pamazen-1b": _stack(128256, 2048, 4, _attn_spec(16, 4, 128, 64, 128),
                         _parallel_spec(32, 8, 64, 1024, 16, 32, 64), 6,
                         _moe(1024, 14, 4, 2, 4, 3, 1024)),
    # layers as wide as an 8B model's
    "pamazen-4k": _stack(32000, 4096, 4, _attn_spec(32, 8, 128, 64, 128),
                         _parallel_spec(64, 8, 64, 2048, 16, 64, 64), 3,
                         _moe(2048, 12, 4, 4, 4, 3, 2048)),
}


def _build(config: Optional[Dict[str, Any]] = None,
           preset: str = "pamazen-tiny",
           overrides: Optional[Dict[str, Any]] = None) -> PamazenForCausalLM:
    raw = dict(config if config is not None else PRESETS[preset])
    raw.update(overrides or {})
    return PamazenForCausalLM(PamazenConfig(raw))


register_token_batch_arch("pamazen", _build, architecture="Pamazen")


@register_arch("pamazen")
def pamazen(preset: str = "pamazen-tiny", config=None,
            **overrides) -> PamazenForCausalLM:
    return _build(config, preset, overrides)
