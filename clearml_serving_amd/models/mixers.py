"""Layers for models that run on flat token batches (ops.lm).

Each layer takes h [T, pad32(width)] -- the residual stream in the matrix
product type -- and a ``TokenBatch`` that says which sequence, position, cache
row and state slot every token has. Sizes and constants are constructor
parameters; ``pack`` fills the padded, merged operands from tensors in
checkpoint layout.
"""

from typing import Callable, Dict, Optional

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
    given (another layer's). ``window`` 0: all earlier tokens. ``q_rank``:
    queries come from a normed latent of that size. ``rot_half``: pair i is
    (i, i + dims/2), else (2i, 2i+1); ``rot_scaling``: YaRN's factor,
    original, fast, slow. ``sink``: a learned term in each head's softmax
    denominator. ``gate``: sigmoid of a projection on the heads' outputs."""

    def __init__(self, width: int, heads: int, dim: int, rot_dim: int,
                 vdim: int, kv_rank: int, scale: float, window: int,
                 rot_base: float, rot_dims: int, eps: float,
                 owns_kv: bool = True, q_rank: Optional[int] = None,
                 rot_half: bool = False,
                 rot_scaling: Optional[Dict[str, float]] = None,
                 sink: bool = True, gate: bool = False):
        super().__init__()
        if q_rank is not None and not owns_kv:
            raise ValueError("a query latent needs a key latent of its own")
        if rot_dims % 2 or not 0 < rot_dims <= rot_dim:
            raise ValueError("rotated dimensions {} of {}".format(rot_dims,
                                                                  rot_dim))
        self.width, self.heads = width, heads
        self.dim, self.rot_dim, self.vdim = dim, rot_dim, vdim
        self.kv_rank, self.scale, self.window = kv_rank, scale, window
        self.eps, self.owns_kv, self.q_rank = eps, owns_kv, q_rank
        self.rot_base, self.rot_dims = rot_base, rot_dims
        self.rot_half, self.rot_scaling = rot_half, rot_scaling
        wp = pad32(width)
        dp, rp = pad32(dim), pad32(rot_dim)
        cp, vp = pad32(kv_rank), pad32(vdim)
        self.dp, self.rp, self.cp, self.vp = dp, rp, cp, vp
        self.q_cols = heads * (dp + rp)
        self.row = cp + rp  # cached elements per token
        # one product of h: [q or its latent | key latent | gate]
        self.q_in = self.q_cols if q_rank is None else pad32(q_rank)
        self.gate_at = self.q_in + (self.row if owns_kv else 0)
        self.qkv = _param(self.gate_at + (heads * vp if gate else 0), wp)
        self.has_gate = gate
        self.q_norm = None if q_rank is None else _param(self.q_in)
        self.uq = None if q_rank is None else _param(self.q_cols, self.q_in)
        self.kv_norm = _param(cp) if owns_kv else None
        self.uk_t = _param(heads, cp, dp)   # absorbs W_uk into the query
        self.uv = _param(heads, vp, cp)
        self.sink = _param(heads) if sink else None
        self.o = _param(wp, heads * vp)
        self.rot: Optional[lm.Rotary] = None
        self.kv_up: Optional[torch.Tensor] = None

    def shapes(self) -> dict:
        h = self.heads
        q_out = h * (self.dim + self.rot_dim)
        out = {"uk": (h * self.dim, self.kv_rank),
               "uv": (h * self.vdim, self.kv_rank),
               "o": (self.width, h * self.vdim)}
        if self.q_rank is None:
            out["q"] = (q_out, self.width)
        else:
            out["dq"] = (self.q_rank, self.width)
            out["dq.norm"] = (self.q_rank,)
            out["uq"] = (q_out, self.q_rank)
        if self.sink is not None:
            out["sink"] = (h,)
        if self.has_gate:
            out["g"] = (h * self.vdim, self.width)
        if self.owns_kv:
            out["dkv"] = (self.kv_rank + self.rot_dim, self.width)
            out["dkv.norm"] = (self.kv_rank,)
        return out

    def pack(self, get: Get) -> None:
        h, dim = self.heads, self.dim

        def heads_of_q(dst, src):  # rows head by head: [unrotated, rotated]
            q = src.view(h, dim + self.rot_dim, -1)
            w = dst.view(h, self.dp + self.rp, -1)
            _fill(w[:, :self.dp], q[:, :dim])
            _fill(w[:, self.dp:], q[:, dim:])

        if self.q_rank is None:
            heads_of_q(self.qkv.data[:self.q_in], get("q"))
        else:
            _fill(self.qkv.data[:self.q_in], get("dq"))
            _fill(self.q_norm.data, get("dq.norm"))
            heads_of_q(self.uq.data, get("uq"))
        if self.owns_kv:
            d = get("dkv")
            w = self.qkv.data[self.q_in:self.gate_at]
            _fill(w[:self.cp], d[:self.kv_rank])
            _fill(w[self.cp:], d[self.kv_rank:])
            _fill(self.kv_norm.data, get("dkv.norm"))
        if self.has_gate:
            _fill(self.qkv.data[self.gate_at:].view(h, self.vp, -1),
                  get("g").view(h, self.vdim, self.width))
        _fill(self.uk_t.data,
              get("uk").view(h, dim, self.kv_rank).transpose(1, 2))
        _fill(self.uv.data, get("uv").view(h, self.vdim, self.kv_rank))
        if self.sink is not None:
            _fill(self.sink.data, get("sink"))
        o = get("o").view(self.width, h, self.vdim)
        _fill(self.o.data.view(-1, h, self.vp), o)

    def finalize(self) -> None:
        """tables and weight layouts that follow from the loaded weights"""
        gain = 1.0
        if self.rot_scaling is None:
            i = torch.arange(self.rot_dims // 2, dtype=torch.float64)
            freq = float(self.rot_base) ** (-2.0 * i / self.rot_dims)
        else:
            s = self.rot_scaling
            freq, gain = lm.yarn_frequencies(
                self.rot_base, self.rot_dims, float(s["factor"]),
                float(s["original"]), float(s["fast"]), float(s["slow"]))
        self.rot = lm.Rotary(freq.to(torch.float32).to(self.qkv.device), gain,
                             self.rot_half)
        # prompts rebuild keys and values: [H*dp | H*vp] rows
        self.kv_up = torch.cat([
            self.uk_t.data.transpose(1, 2).reshape(-1, self.cp),
            self.uv.data.reshape(-1, self.cp)])

    def can_expand(self) -> bool:
        """whether ops.lm.latent_prompt takes this head size"""
        return (self.dp + self.rp <= lm.PROMPT_MAX_HEAD
                and self.vp <= lm.PROMPT_MAX_HEAD)

    def _queries(self, z, batch, cache, n):
        """Rotate, norm and store what the merged product z holds.
        -> (q [T, heads x (dp | rp)], rotated behind the first n tokens;
        q_abs [n, heads, row], complete)"""
        q_abs = z.new_empty(n, self.heads, self.row) if n else None
        if self.q_rank is None:
            q = z[:, :self.q_cols]
            lm.latent_prep(z[:, :self.gate_at], batch.positions,
                           batch.slot_mapping, self.rot, self.heads, self.dp,
                           self.rp, self.cp, self.kv_rank, self.eps,
                           self.kv_norm, cache if self.owns_kv else None,
                           q_abs)
            if n:
                lm.head_gemm(q.unflatten(1, (self.heads, -1))
                             [:n, :, :self.dp], self.uk_t,
                             q_abs[..., :self.cp])
            return q, q_abs
        cq = lm.latent_prep_two(
            z[:, :self.q_in], z[:, self.q_in:self.gate_at], batch.positions,
            batch.slot_mapping, self.rot, self.rp, self.cp, self.kv_rank,
            self.q_rank, self.eps, self.q_norm, self.kv_norm, cache)
        q = linear(cq, self.uq)
        if n:
            lm.absorb_query(q.unflatten(1, (self.heads, -1))[:n], self.uk_t,
                            q_abs, batch.positions, self.rot)
        if n < q.shape[0]:
            lm.rotate_query(q[n:], batch.positions[n:], self.rot, self.heads,
                            self.dp, self.rp)
        return q, q_abs

    def forward(self, h, batch, cache):
        t, n = h.shape[0], batch.n_abs
        z = linear(h, self.qkv)
        q, q_abs = self._queries(z, batch, cache, n)
        gate = z[:, self.gate_at:] if self.has_gate else None
        ctx = h.new_empty(t, self.heads, self.vp)
        if n:
            lat = lm.latent_attention(
                q_abs, cache, batch.block_table, batch.tok_seq,
                batch.positions, self.sink, self.scale, self.window, self.cp,
                batch.max_keys)
            lm.head_gemm(lat, self.uv, ctx[:n],
                         None if gate is None else gate[:n])
        if n < t:
            kv_rows, qtiles = batch.prompts[self.window]
            rows = lm.gather_rows(cache, kv_rows)
            kv = linear(rows[:, :self.cp], self.kv_up)
            lm.latent_prompt(q, kv, rows, self.sink, qtiles, ctx,
                             self.heads, self.dp, self.rp, self.cp, self.vp,
                             self.window, self.scale, gate)
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
    """down(act(gate h + b) * (up h + b)); ``act``: gelu_tanh or silu. The
    bias of ``down`` is ``down_b``, added by the norm that follows; without
    ``bias`` there are none."""

    def __init__(self, width: int, ff: int, act: str = "gelu_tanh",
                 bias: bool = True):
        super().__init__()
        self.width, self.ff, self.act = width, ff, act
        w, f = pad32(width), pad32(ff)
        self.fp = f
        self.gate_up = _param(2 * f, w)
        self.gate_up_b = _param(2 * f) if bias else None
        self.down = _param(w, f)
        self.down_b = _param(w) if bias else None

    def shapes(self) -> dict:
        out = {"gate": (self.ff, self.width), "up": (self.ff, self.width),
               "down": (self.width, self.ff)}
        if self.down_b is not None:
            out.update({"gate.b": (self.ff,), "up.b": (self.ff,),
                        "down.b": (self.width,)})
        return out

    def pack(self, get: Get) -> None:
        for half, name in enumerate(("gate", "up")):
            _fill(self.gate_up.data.view(2, self.fp, -1)[half], get(name))
            if self.gate_up_b is not None:
                _fill(self.gate_up_b.data.view(2, -1)[half],
                      get(name + ".b"))
        _fill(self.down.data, get("down"))
        if self.down_b is not None:
            _fill(self.down_b.data, get("down.b"))

    def forward(self, h):
        return linear(lm.gated_mul(linear(h, self.gate_up), self.gate_up_b,
                                   self.act), self.down)


class ExpertMlp(nn.Module):
    """Of ``experts`` feed-forwards down(act(up h)) each token takes the
    ``top`` with the largest router logits, weighed by the softmax over
    those (csrc/lm/moe.hip). The weighted sum is left to the norm that
    follows: forward -> (rows of all slots, (pos, share))."""

    def __init__(self, width: int, ff: int, experts: int, top: int,
                 act: str = "relu2"):
        super().__init__()
        if not 1 <= top <= experts:
            raise ValueError("{} of {} experts".format(top, experts))
        self.width, self.ff, self.act = width, ff, act
        self.experts, self.top = experts, top
        w, f = pad32(width), pad32(ff)
        self.router = _param(experts, w)
        self.up = _param(experts, f, w)
        self.down = _param(experts, w, f)

    def shapes(self) -> dict:
        out = {"router": (self.experts, self.width)}
        for e in range(self.experts):
            out["e{}.up".format(e)] = (self.ff, self.width)
            out["e{}.down".format(e)] = (self.width, self.ff)
        return out

    def pack(self, get: Get) -> None:
        _fill(self.router.data, get("router"))
        for e in range(self.experts):
            _fill(self.up.data[e], get("e{}.up".format(e)))
            _fill(self.down.data[e], get("e{}.down".format(e)))

    def forward(self, h):
        rows = lm.expert_tile_rows(
            h.shape[0], self.experts, self.top, h.dtype,
            (self.up.shape[2], self.down.shape[2]))
        plan = lm.moe_route(h, self.router, self.top, rows)
        hidden = lm.moe_gemm(h, self.up, plan, self.act, gather=True)
        out = lm.moe_gemm(hidden, self.down, plan, "none", gather=False)
        return out, (plan.pos, plan.share)
