"""Layers for models that run on flat token batches (ops.lm).

Each layer takes h [T, pad32(width)] -- the residual stream in the matrix
product type -- and a ``TokenBatch`` that says which sequence, position, cache
row and state slot every token has. Sizes and constants are constructor
parameters; ``pack`` fills the padded, merged operands from tensors in
checkpoint layout.
"""

from typing import Callable, List, Optional

import torch
import torch.nn as nn

from .. import ops
from ..ops import lm
from ..ops.lm import pad32

Get = Callable[[str], torch.Tensor]


def _param(*shape) -> nn.Parameter:
    return nn.Parameter(torch.zeros(*shape), requires_grad=False)


def _fill(dst: torch.Tensor, src: torch.Tensor) -> None:
    """leading corner of dst = src, the padding stays zero"""
    dst[tuple(slice(0, n) for n in src.shape)] = src.to(dst.dtype)


def linear(x: torch.Tensor, w: torch.Tensor) -> torch.Tensor:
    """decode-sized batches take the in-tree MFMA kernel, others hipBLASLt"""
    return ops.skinny_linear(x, w)


class LatentAttention(nn.Module):
    """Attention on a cached latent shared by all heads (csrc/lm/latent.hip).

    ``owns_kv=False``: no latent of its own, attends to the cache it is
    given (another layer's). ``window`` 0: all earlier tokens."""

    def __init__(self, width: int, heads: int, dim: int, rot_dim: int,
                 vdim: int, kv_rank: int, scale: float, window: int,
                 rot_base: float, rot_dims: int, eps: float,
                 owns_kv: bool = True):
        super().__init__()
        self.width, self.heads = width, heads
        self.dim, self.rot_dim, self.vdim = dim, rot_dim, vdim
        self.kv_rank, self.scale, self.window = kv_rank, scale, window
        self.eps, self.owns_kv = eps, owns_kv
        self.rot_base, self.rot_dims = rot_base, rot_dims
        wp = pad32(width)
        dp, rp = pad32(dim), pad32(rot_dim)
        cp, vp = pad32(kv_rank), pad32(vdim)
        self.dp, self.rp, self.cp, self.vp = dp, rp, cp, vp
        self.q_cols = heads * (dp + rp)
        self.row = cp + rp  # cached elements per token
        self.qkv = _param(self.q_cols + (self.row if owns_kv else 0), wp)
        self.kv_norm = _param(cp) if owns_kv else None
        self.uk_t = _param(heads, cp, dp)   # absorbs W_uk into the query
        self.uv = _param(heads, vp, cp)
        self.sink = _param(heads)
        self.o = _param(wp, heads * vp)
        self.inv_freq: Optional[torch.Tensor] = None
        self.kv_up: Optional[torch.Tensor] = None

    def names(self) -> List[str]:
        own = ["dkv", "dkv.norm"] if self.owns_kv else []
        return ["q", *own, "uk", "uv", "sink", "o"]

    def shapes(self) -> dict:
        h = self.heads
        out = {"q": (h * (self.dim + self.rot_dim), self.width),
               "uk": (h * self.dim, self.kv_rank),
               "uv": (h * self.vdim, self.kv_rank),
               "sink": (h,), "o": (self.width, h * self.vdim)}
        if self.owns_kv:
            out["dkv"] = (self.kv_rank + self.rot_dim, self.width)
            out["dkv.norm"] = (self.kv_rank,)
        return out

    def pack(self, get: Get) -> None:
        h, dim = self.heads, self.dim
        q = get("q").view(h, dim + self.rot_dim, self.width)
        w = self.qkv.data[:self.q_cols].view(h, self.dp + self.rp, -1)
        _fill(w[:, :self.dp], q[:, :dim])
        _fill(w[:, self.dp:], q[:, dim:])
        if self.owns_kv:
            d = get("dkv")
            w = self.qkv.data[self.q_cols:]
            _fill(w[:self.cp], d[:self.kv_rank])
            _fill(w[self.cp:], d[self.kv_rank:])
            _fill(self.kv_norm.data, get("dkv.norm"))
        _fill(self.uk_t.data,
              get("uk").view(h, dim, self.kv_rank).transpose(1, 2))
        _fill(self.uv.data, get("uv").view(h, self.vdim, self.kv_rank))
        _fill(self.sink.data, get("sink"))
        o = get("o").view(self.width, h, self.vdim)
        _fill(self.o.data.view(-1, h, self.vp), o)

    def finalize(self) -> None:
        """tables and weight layouts that follow from the loaded weights"""
        dev = self.qkv.device
        i = torch.arange(self.rot_dims // 2, dtype=torch.float64)
        self.inv_freq = (float(self.rot_base) ** (
            -2.0 * i / self.rot_dims)).to(torch.float32).to(dev)
        # prompts rebuild keys and values: [H*dp | H*vp] rows
        self.kv_up = torch.cat([
            self.uk_t.data.transpose(1, 2).reshape(-1, self.cp),
            self.uv.data.reshape(-1, self.cp)])

    def can_expand(self) -> bool:
        """whether ops.lm.latent_prompt takes this head size"""
        return (self.dp + self.rp <= lm.PROMPT_MAX_HEAD
                and self.vp <= lm.PROMPT_MAX_HEAD)

    def forward(self, h, batch, cache):
        t = h.shape[0]
        qkv = linear(h, self.qkv)
        n = batch.n_abs
        q = qkv[:, :self.q_cols].unflatten(1, (self.heads, -1))
        q_abs = h.new_empty(n, self.heads, self.row) if n else None
        lm.latent_prep(qkv, batch.positions, batch.slot_mapping,
                       self.inv_freq, self.heads, self.dp, self.rp, self.cp,
                       self.kv_rank, self.eps, self.kv_norm,
                       cache if self.owns_kv else None, q_abs)
        ctx = h.new_empty(t, self.heads, self.vp)
        if n:
            lm.head_gemm(q[:n, :, :self.dp], self.uk_t, q_abs[..., :self.cp])
            lat = lm.latent_attention(
                q_abs, cache, batch.block_table, batch.tok_seq,
                batch.positions, self.sink, self.scale, self.window, self.cp,
                batch.max_keys)
            lm.head_gemm(lat, self.uv, ctx[:n])
        if n < t:
            kv_rows, qtiles = batch.prompts[self.window]
            rows = lm.gather_rows(cache, kv_rows)
            kv = linear(rows[:, :self.cp], self.kv_up)
            lm.latent_prompt(qkv, kv, rows, self.sink, qtiles, ctx,
                             self.heads, self.dp, self.rp, self.cp, self.vp,
                             self.window, self.scale)
        return linear(ctx.view(t, -1), self.o)


class RgLru(nn.Module):
    """Gated branch times a real-gated linear recurrence behind a causal
    convolution (csrc/lm/rglru.hip)."""

    def __init__(self, width: int, channels: int, blocks: int, taps: int):
        super().__init__()
        if channels % blocks:
            raise ValueError("recurrence width {} is not a multiple of its "
                             "{} blocks".format(channels, blocks))
        self.width, self.channels = width, channels
        self.blocks, self.taps = blocks, taps
        self.bw = channels // blocks
        self.bp = pad32(self.bw)
        self.wp = self.bp * blocks
        w = pad32(width)
        self.yx = _param(2 * self.wp, w)
        self.yx_b = _param(2 * self.wp)
        self.conv = _param(taps, self.wp)
        self.conv_b = _param(self.wp)
        self.ra = _param(blocks, self.bp, self.bp)
        self.ri = _param(blocks, self.bp, self.bp)
        self.ra_b = _param(self.wp)
        self.ri_b = _param(self.wp)
        self.lam = _param(self.wp)
        self.o = _param(w, self.wp)
        self._w = None

    def shapes(self) -> dict:
        c, b, k, w = self.channels, self.blocks, self.bw, self.width
        return {"y": (c, w), "y.b": (c,), "x": (c, w), "x.b": (c,),
                "conv": (c, self.taps), "conv.b": (c,),
                "ra": (b, k, k), "ra.b": (b, k), "ri": (b, k, k),
                "ri.b": (b, k), "lam": (c,), "o": (w, c)}

    def pack(self, get: Get) -> None:
        b, k = self.blocks, self.bw

        def vec(dst, src):  # [channels] -> blocks of bp
            _fill(dst.view(b, self.bp), src.reshape(b, k))

        for half, name in enumerate(("y", "x")):
            w = self.yx.data.view(2, b, self.bp, -1)[half]
            _fill(w, get(name).view(b, k, self.width))
            vec(self.yx_b.data.view(2, -1)[half], get(name + ".b"))
        _fill(self.conv.data.view(self.taps, b, self.bp),
              get("conv").t().reshape(self.taps, b, k))
        vec(self.conv_b.data, get("conv.b"))
        _fill(self.ra.data, get("ra"))
        _fill(self.ri.data, get("ri"))
        vec(self.ra_b.data, get("ra.b"))
        vec(self.ri_b.data, get("ri.b"))
        vec(self.lam.data, get("lam"))
        _fill(self.o.data.view(-1, b, self.bp),
              get("o").view(self.width, b, k))

    def finalize(self) -> None:
        self._w = lm.RglruWeights(
            self.yx_b.data, self.conv.data, self.conv_b.data, self.ra.data,
            self.ra_b.data, self.ri.data, self.ri_b.data, self.lam.data)

    def forward(self, h, batch, cache):
        state, ring = cache
        yx = linear(h, self.yx)
        out = h.new_empty(h.shape[0], self.wp)
        lm.rglru_step(yx, self._w, state, ring, batch.positions,
                      batch.state_slots, out, batch.n_single)
        lm.rglru_prefill(yx, self._w, state, ring, batch.tiles, batch.seqs,
                         out, batch.tile)
        return linear(out, self.o)


class GatedMlp(nn.Module):
    """down(gelu_tanh(gate h + b) * (up h + b)); the bias of ``down`` is
    ``down_b``, added by the norm that follows."""

    def __init__(self, width: int, ff: int):
        super().__init__()
        self.width, self.ff = width, ff
        w, f = pad32(width), pad32(ff)
        self.fp = f
        self.gate_up = _param(2 * f, w)
        self.gate_up_b = _param(2 * f)
        self.down = _param(w, f)
        self.down_b = _param(w)

    def shapes(self) -> dict:
        return {"gate": (self.ff, self.width), "gate.b": (self.ff,),
                "up": (self.ff, self.width), "up.b": (self.ff,),
                "down": (self.width, self.ff), "down.b": (self.width,)}

    def pack(self, get: Get) -> None:
        for half, name in enumerate(("gate", "up")):
            _fill(self.gate_up.data.view(2, self.fp, -1)[half], get(name))
            _fill(self.gate_up_b.data.view(2, -1)[half], get(name + ".b"))
        _fill(self.down.data, get("down"))
        _fill(self.down_b.data, get("down.b"))

    def forward(self, h):
        return linear(lm.gelu_mul(linear(h, self.gate_up), self.gate_up_b),
                      self.down)
