"""Layers for models that run on flat token batches (ops.lm).

Each layer takes h [T, pad32(width)] -- the residual stream in the matrix
product type -- and a ``TokenBatch`` that says which sequence, position, cache
row and state slot every token has. Sizes and constants are constructor
parameters; ``pack`` fills the padded, merged operands from tensors in
checkpoint layout.
"""

from typing import Callable, Dict, List, Optional, Tuple, Union

import torch
import torch.nn as nn

from .. import ops
from ..ops import delta, grouped, linear_state, lm
from ..ops.lm import pad32

Get = Callable[[str], torch.Tensor]


def _param(*shape) -> nn.Parameter:
    return nn.Parameter(torch.zeros(shape), requires_grad=False)


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

    @property
    def view(self):
        """what a query sees, as TokenBatch names it"""
        return self.window

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


class GroupedAttention(nn.Module):
    """Grouped-query attention (csrc/lm/gqa.hip): ``heads`` query heads on
    ``kv_heads`` cached key/value heads.

    ``rot``: (base, rotated dimensions, factor that divides the frequencies),
    pairs (2i, 2i+1) or, ``rot_half``, (i, i + dimensions/2), or None.
    ``window`` 0: all earlier tokens; else the last ``window`` and the first
    ``keep`` ones, or in front of the window the mean key and value of every
    whole block of ``pool`` tokens. ``cap``: scores become cap * tanh(score /
    cap). ``qk_norm``: norm of queries and keys, "head" (or True) one by one,
    "all" over all heads at once. ``bias``: on queries, keys and values.
    ``values_are_keys``: no projection of their own, the keys before norm and
    rotation. ``sink``: "learned" term per head in the softmax's denominator,
    "one" (a learned term of 0) or None. ``v_mix``: values mixed with those of
    the first layer that does."""

    def __init__(self, width: int, heads: int, kv_heads: int, dim: int,
                 vdim: int, scale: float, eps: float = 0.0,
                 rot: Optional[Tuple[float, int, float]] = None,
                 window: int = 0, keep: int = 0, cap: float = 0.0,
                 qk_norm: Union[bool, str] = False,
                 values_are_keys: bool = False, sink: Optional[str] = None,
                 v_mix: bool = False, rot_half: bool = False, pool: int = 0,
                 bias: bool = False):
        super().__init__()
        if kv_heads < 1 or heads % kv_heads:
            raise ValueError("{} query heads on {} key/value heads".format(
                heads, kv_heads))
        if rot is not None and (rot[1] % 2 or not 0 < rot[1] <= dim):
            raise ValueError("rotated dimensions {} of {}".format(
                rot[1], dim))
        if values_are_keys and (vdim != dim or v_mix or rot is not None):
            raise ValueError("values that are keys have the keys' size and "
                             "go with neither mixing nor rotation")
        if (keep or pool) and not window:
            raise ValueError("kept tokens or pooled blocks without a window")
        if keep and pool:
            raise ValueError("kept tokens beside pooled blocks")
        whole = qk_norm == "all"
        if values_are_keys and (whole or pool or bias):
            raise ValueError("values that are keys go with neither pooled "
                             "blocks, biases nor a norm over all heads")
        if sink not in (None, "one", "learned"):
            raise ValueError("unknown sink '{}'".format(sink))
        self.width, self.heads, self.kv_heads = width, heads, kv_heads
        self.dim, self.vdim, self.eps = dim, vdim, eps
        self.rot_spec, self.v_mix, self.lam = rot, v_mix, 0.0
        self.kp, self.vp = pad32(dim), pad32(vdim)
        self.spec = grouped.GroupedSpec(
            heads, kv_heads, self.kp, self.vp, dim, values_are_keys, window,
            keep, scale, cap, 1.0, pool, whole)
        # one product of h: [queries | keys | values]
        self.k_at = heads * self.kp
        self.v_at = self.k_at + kv_heads * self.kp
        self.cols = self.v_at + (0 if values_are_keys else
                                 kv_heads * self.vp)
        self.q_norm = self.k_norm = None
        if qk_norm:
            self.q_norm = _param(self.kp * (heads if whole else 1))
            self.k_norm = _param(self.kp * (kv_heads if whole else 1))
        self.bias = _param(self.cols) if bias else None
        # the kernels rotate neighbours: halves are brought together when
        # weights are packed (scores do not depend on the channels' order)
        self.order = None
        if rot_half and rot is not None:
            self.order = torch.arange(dim)
            self.order[:rot[1]] = self.order[:rot[1]].view(2, -1).t() \
                .reshape(-1)
        self.sink_kind = sink
        self.sink = None if sink is None else _param(heads)
        self.vmix = _param() if v_mix else None
        self.rot: Optional[lm.Rotary] = None

    @property
    def view(self):
        """what a query sees, as TokenBatch names it"""
        s = self.spec
        if s.pool:
            return s.window, 0, s.pool
        return (s.window, s.keep) if s.keep else s.window

    @property
    def out_cols(self) -> int:
        return self.heads * self.vp

    def scaled(self, out_scale: float) -> "GroupedAttention":
        """the result times a constant"""
        self.spec = self.spec._replace(out_scale=out_scale)
        return self

    def shapes(self) -> dict:
        h, g = self.heads, self.kv_heads
        out = {"q": (h * self.dim, self.width),
               "k": (g * self.dim, self.width),
               "o": (self.width, h * self.vdim)}
        if not self.spec.same:
            out["v"] = (g * self.vdim, self.width)
        if self.q_norm is not None:
            n = (h, g) if self.spec.whole else (1, 1)
            out["q.norm"], out["k.norm"] = ((m * self.dim,) for m in n)
        if self.bias is not None:
            for name in "qkv":
                out[name + ".b"] = out[name][:1]
        if self.sink_kind == "learned":
            out["sink"] = (h,)
        if self.v_mix:
            out["vmix"] = ()
        return out

    def _channels(self, dst: torch.Tensor, src: torch.Tensor, n: int,
                  name: str) -> None:
        """n heads' channels, in the kernels' order"""
        src = src.reshape(n, src.shape[0] // n, -1)
        if self.order is not None and name != "v":
            src = src[:, self.order]
        _fill(dst.view(n, dst.shape[0] // n, -1), src)

    def _parts(self):
        parts = [("q", 0, self.heads, self.kp),
                 ("k", self.k_at, self.kv_heads, self.kp)]
        if not self.spec.same:
            parts.append(("v", self.v_at, self.kv_heads, self.vp))
        return parts

    def pack_in(self, w: torch.Tensor, get: Get) -> None:
        """rows of the product of h"""
        for name, at, n, size in self._parts():
            self._channels(w[at:at + n * size], get(name), n, name)

    def pack_out(self, w: torch.Tensor, get: Get) -> None:
        """columns of the product of the heads' results"""
        _fill(w.view(w.shape[0], self.heads, self.vp),
              get("o").view(self.width, self.heads, self.vdim))

    def pack_own(self, get: Get) -> None:
        if self.q_norm is not None:
            n = (self.heads, self.kv_heads) if self.spec.whole else (1, 1)
            self._channels(self.q_norm.data, get("q.norm"), n[0], "q")
            self._channels(self.k_norm.data, get("k.norm"), n[1], "k")
        if self.bias is not None:
            for name, at, n, size in self._parts():
                self._channels(self.bias.data[at:at + n * size],
                               get(name + ".b"), n, name)
        if self.sink_kind == "learned":
            _fill(self.sink.data, get("sink"))
        if self.v_mix:
            _fill(self.vmix.data, get("vmix"))

    def finalize(self, device) -> None:
        if self.rot_spec is not None:
            base, dims, factor = self.rot_spec
            i = torch.arange(dims // 2, dtype=torch.float64)
            freq = float(base) ** (-2.0 * i / dims) / factor
            self.rot = lm.Rotary(freq.to(torch.float32).to(device))
        if self.v_mix:
            self.lam = float(self.vmix)

    def can_expand(self) -> bool:
        """whether prompts take tiles of queries (ops.grouped.prompt)"""
        return max(self.kp, self.vp) <= lm.PROMPT_MAX_HEAD

    def values(self, z) -> torch.Tensor:
        return z[:, self.v_at:self.cols]

    def page_layout(self) -> tuple:
        s = self.spec
        return ("paged", s.row, s.pool) if s.pool else ("paged", s.row)

    def attend(self, z, batch, cache, out, first=None):
        """z [T, >= cols]: the product of h; out [T, out_cols]. ``first``:
        the values that this layer's are mixed with"""
        t, n, s = z.shape[0], batch.n_abs, self.spec
        grouped.prepare(z, self.k_at, self.v_at, batch.positions,
                        batch.slot_mapping, self.rot, s, self.q_norm,
                        self.k_norm, self.eps, first, self.lam, cache,
                        self.bias)
        if s.pool:
            grouped.pool_rows(cache, batch.block_table, batch.tok_seq,
                              batch.positions, s.pool)
        q = z[:, :self.k_at]
        if n:
            grouped.attention(q, cache, batch.block_table, batch.tok_seq,
                              batch.positions, self.sink, out, n, s,
                              batch.max_keys)
        if n < t:
            rows, qtiles = batch.prompts[self.view]
            grouped.prompt(q, lm.gather_rows(cache, rows), self.sink, qtiles,
                           out, s)


class GroupedAttentionMixer(nn.Module):
    """GroupedAttention as a layer's mixer."""

    def __init__(self, width: int, *args, **kw):
        super().__init__()
        self.attn = a = GroupedAttention(width, *args, **kw)
        wp = pad32(width)
        self.qkv = _param(a.cols, wp)
        self.o = _param(wp, a.out_cols)

    def shapes(self) -> dict:
        return self.attn.shapes()

    def pack(self, get: Get) -> None:
        self.attn.pack_in(self.qkv.data, get)
        self.attn.pack_out(self.o.data, get)
        self.attn.pack_own(get)

    def finalize(self) -> None:
        self.attn.finalize(self.qkv.device)

    def cache_layout(self) -> tuple:
        return self.attn.page_layout()

    def forward(self, h, batch, cache, carry):
        """``carry``: what layers of one forward hand on ("values")"""
        a, first = self.attn, None
        z = linear(h, self.qkv)
        if a.v_mix:
            first = carry.get("values")
            if first is None:  # this is the first such layer
                carry["values"] = a.values(z)
        ctx = h.new_empty(h.shape[0], a.out_cols)
        a.attend(z, batch, cache, ctx, first)
        return linear(ctx, self.o)


class DeltaRule(nn.Module):
    """Generalised delta rule (csrc/lm/delta.hip): a float state per head with
    decay per key channel, a removal term along the unit key, and outputs that
    are normed per head and gated. ``rank``: inner size of the decay's
    projection, which a checkpoint's tensors tell (``fit``)."""

    def __init__(self, width: int, heads: int, dim: int, eps: float,
                 rank: int = 64):
        super().__init__()
        self.width, self.heads, self.dim, self.eps = width, heads, dim, eps
        self.dp = delta.head_pad(dim)
        n = heads * self.dp
        self.ab, self.w0, self.norm = _param(n), _param(n), _param(n)
        self.out_scale = 1.0
        self._set_rank(rank)

    def _set_rank(self, rank: int) -> None:
        self.rank, self.rp = rank, pad32(rank)
        n = self.heads * self.dp
        self.w2 = _param(n, self.rp)
        # one product of h: [r | k | v | g | a | low-rank input of the decay]
        self.cols = 5 * n + self.rp
        self._w: Optional[delta.DeltaWeights] = None

    @property
    def out_cols(self) -> int:
        return self.heads * self.dp

    def scaled(self, out_scale: float) -> "DeltaRule":
        """the result times a constant"""
        self.out_scale = out_scale
        return self

    def fit(self, get: Get) -> None:
        rank = get("w1").shape[0]
        if rank != self.rank:
            self._set_rank(rank)

    def shapes(self) -> dict:
        n, w = self.heads * self.dim, self.width
        out = {k: (n, w) for k in "rkvga"}
        out.update({"a.b": (n,), "w0": (n,), "norm": (n,),
                    "w1": (self.rank, w), "w2": (n, self.rank), "o": (w, n)})
        return out

    def _heads(self, dst: torch.Tensor, src: torch.Tensor) -> None:
        _fill(dst.view(self.heads, self.dp, -1),
              src.reshape(self.heads, self.dim, -1))

    def pack_in(self, w: torch.Tensor, get: Get) -> None:
        n = self.heads * self.dp
        for i, name in enumerate("rkvga"):
            self._heads(w[i * n:(i + 1) * n], get(name))
        _fill(w[5 * n:5 * n + self.rp], get("w1"))

    def pack_out(self, w: torch.Tensor, get: Get) -> None:
        _fill(w.view(w.shape[0], self.heads, self.dp),
              get("o").view(self.width, self.heads, self.dim))

    def pack_own(self, get: Get) -> None:
        self._heads(self.w2.data, get("w2"))
        for dst, name in ((self.ab, "a.b"), (self.w0, "w0"),
                          (self.norm, "norm")):
            self._heads(dst.data, get(name))

    def finalize(self) -> None:
        self._w = delta.DeltaWeights(self.w2.data, self.w0.data,
                                     self.ab.data, self.norm.data)

    def state_layout(self) -> tuple:
        return "state", (self.heads, self.dp, self.dp)

    def scan(self, z, batch, state, out) -> None:
        """z [T, cols]: the product of h; out [T, out_cols]"""
        n = self.heads * self.dp
        delta.delta_rule(z, tuple(i * n for i in range(6)), self._w, state,
                         batch.positions, batch.state_slots, batch.seqs, out,
                         batch.n_single, self.dim, self.eps, self.out_scale,
                         batch.tiles.shape[0], batch.tile)


class LinearState(nn.Module):
    """A recurrence with one decay per head behind short convolutions
    (ops/linear_state.py). Subclasses say how a checkpoint names its parts."""

    def __init__(self, width: int, spec: linear_state.StateSpec, skip: bool,
                 conv_bias: bool):
        super().__init__()
        s = self.spec = spec
        if s.groups < 1 or s.heads % s.groups:
            raise ValueError("{} heads on {} groups of keys".format(
                s.heads, s.groups))
        if not 1 <= s.taps <= linear_state.MAX_TAPS:
            raise ValueError("convolution over {} tokens, 1 to {} are "
                             "possible".format(s.taps, linear_state.MAX_TAPS))
        if s.parts < 1 or s.heads * s.vdim % s.parts:
            raise ValueError("norm of {} channels in {} parts".format(
                s.heads * s.vdim, s.parts))
        self.width, self.cols = width, s.cols
        self.out_cols = s.heads * s.vp
        self.conv = _param(s.taps, s.channels)
        self.conv_b = _param(s.channels) if conv_bias else None
        self.a_log, self.dt_bias = _param(s.heads), _param(s.heads)
        self.skip = _param(s.heads) if skip else None
        self.norm = _param(self.out_cols)
        self._w: Optional[linear_state.StateWeights] = None

    # (place, heads, padded and true channels of a head) of q, k, v, gate
    def _places(self):
        s = self.spec
        return {"q": (0, s.groups, s.kp, s.dim),
                "k": (s.k_at, s.groups, s.kp, s.dim),
                "v": (s.v_at, s.heads, s.vp, s.vdim),
                "gate": (s.channels, s.heads, s.vp, s.vdim)}

    def _put(self, dst: torch.Tensor, part: str, src: torch.Tensor) -> None:
        """src [heads * channels, ...] into the part's padded rows of dst"""
        at, n, pad, size = self._places()[part]
        _fill(dst[at:at + n * pad].view(n, pad, -1), src.reshape(n, size, -1))

    def _put_taps(self, part: str, src: torch.Tensor) -> None:
        at, n, pad, size = self._places()[part]
        _fill(self.conv.data[:, at:at + n * pad].view(-1, n, pad),
              src.t().reshape(-1, n, size))

    def pack_out(self, w: torch.Tensor, get: Get) -> None:
        s = self.spec
        _fill(w.view(w.shape[0], s.heads, s.vp),
              get("o").view(self.width, s.heads, s.vdim))

    def finalize(self) -> None:
        def data(p):
            return None if p is None else p.data

        self._w = linear_state.StateWeights(
            self.conv.data, data(self.conv_b), self.a_log.data,
            self.dt_bias.data, data(self.skip), self.norm.data)

    def state_layout(self) -> tuple:
        return self.spec.layout()

    def scan(self, z, batch, state, ring, out) -> None:
        """z [T, cols]: the product of h; out [T, out_cols]"""
        linear_state.linear_state(
            z, self.spec, self._w, state, ring, batch.positions,
            batch.state_slots, batch.tiles, batch.seqs, batch.tile,
            batch.n_single, out)


class GatedDelta(LinearState):
    """Gated delta rule: ``heads`` states of dim x vdim, on ``kv_heads``
    queries and keys."""

    def __init__(self, width: int, heads: int, kv_heads: int, dim: int,
                 vdim: int, taps: int, eps: float):
        super().__init__(width, linear_state.StateSpec(
            True, heads, kv_heads, dim, vdim, taps, heads, eps), False, False)

    def shapes(self) -> dict:
        s, w = self.spec, self.width
        qk, v = s.groups * s.dim, s.heads * s.vdim
        out = {"q": (qk, w), "k": (qk, w), "v": (v, w), "g": (v, w),
               "a": (s.heads, w), "b": (s.heads, w), "o": (w, v),
               "A_log": (s.heads,), "dt_bias": (s.heads,),
               "norm": (s.vdim,)}
        out.update({k + ".conv": (out[k][0], s.taps) for k in "qkv"})
        return out

    def pack_in(self, w: torch.Tensor, get: Get) -> None:
        s = self.spec
        for part, name in (("q", "q"), ("k", "k"), ("v", "v"), ("gate", "g")):
            self._put(w, part, get(name))
        _fill(w[s.a_at:s.a_at + s.sp], get("a"))
        _fill(w[s.a_at + s.sp:], get("b"))

    def pack_own(self, get: Get) -> None:
        for part in "qkv":
            self._put_taps(part, get(part + ".conv"))
        _fill(self.a_log.data, get("A_log"))
        _fill(self.dt_bias.data, get("dt_bias"))
        s = self.spec
        _fill(self.norm.data.view(s.heads, s.vp),
              get("norm").expand(s.heads, -1))


class StateSpace(LinearState):
    """State-space recurrence: ``heads`` states of ``state`` x vdim whose
    inputs and read-outs ``groups`` of heads share; what the norm sees is
    gated already, and cut into ``parts``."""

    def __init__(self, width: int, heads: int, vdim: int, state: int,
                 groups: int, taps: int, parts: int, eps: float):
        super().__init__(width, linear_state.StateSpec(
            False, heads, groups, state, vdim, taps, parts, eps), True, True)

    def shapes(self) -> dict:
        s, w = self.spec, self.width
        inner, gn = s.heads * s.vdim, s.groups * s.dim
        return {"in": (2 * inner + 2 * gn + s.heads, w),
                "conv": (inner + 2 * gn, s.taps),
                "conv.b": (inner + 2 * gn,), "A_log": (s.heads,),
                "dt_bias": (s.heads,), "D": (s.heads,), "norm": (inner,),
                "o": (w, inner)}

    def _split(self, t: torch.Tensor, gate: bool) -> Dict[str, torch.Tensor]:
        """a checkpoint's rows [gate | v | k | q | rest] by part"""
        s = self.spec
        inner, gn = s.heads * s.vdim, s.groups * s.dim
        sizes = ([inner] if gate else []) + [inner, gn, gn]
        names = (["gate"] if gate else []) + ["v", "k", "q"]
        rest = t.shape[0] - sum(sizes)
        return dict(zip(names + ["rest"], torch.split(t, sizes + [rest])))

    def pack_in(self, w: torch.Tensor, get: Get) -> None:
        parts = self._split(get("in"), True)
        _fill(w[self.spec.a_at:], parts.pop("rest"))
        for part, src in parts.items():
            self._put(w, part, src)

    def pack_own(self, get: Get) -> None:
        parts = self._split(get("conv"), False)
        parts.pop("rest")
        for part, src in parts.items():
            self._put_taps(part, src)
        parts = self._split(get("conv.b"), False)
        parts.pop("rest")
        for part, src in parts.items():
            self._put(self.conv_b.data, part, src)
        for dst, name in ((self.a_log, "A_log"), (self.dt_bias, "dt_bias"),
                          (self.skip, "D")):
            _fill(dst.data, get(name))
        s = self.spec
        _fill(self.norm.data.view(s.heads, s.vp),
              get("norm").view(s.heads, s.vdim))


class RecurrentMixer(nn.Module):
    """A recurrence as a layer's mixer. Its output product is the layer's,
    which can take the feed-forward's along."""

    def __init__(self, width: int, scan: LinearState):
        super().__init__()
        self.rec = scan
        self.inp = _param(scan.cols, pad32(width))

    @property
    def out_cols(self) -> int:
        return self.rec.out_cols

    def shapes(self) -> dict:
        return self.rec.shapes()

    def pack(self, get: Get) -> None:
        self.rec.pack_in(self.inp.data, get)
        self.rec.pack_own(get)

    def pack_out(self, w: torch.Tensor, get: Get) -> None:
        self.rec.pack_out(w, get)

    def finalize(self) -> None:
        self.rec.finalize()

    def cache_layout(self) -> tuple:
        return self.rec.state_layout()

    def context(self, h, batch, cache, out) -> None:
        """what the output product reads, into out [T, out_cols]"""
        self.rec.scan(linear(h, self.inp), batch, *cache, out)


class ParallelMixer(nn.Module):
    """Two mixers that read the same input; the result is their weighted sum.
    Both inputs are one product, and both outputs another. ``norm_outputs``:
    each output has a product of its own and, before the sum, a norm, which is
    left to the kernel that adds them up (``branches``)."""

    def __init__(self, width: int, left: GroupedAttention, left_scale: float,
                 right: Union[DeltaRule, LinearState], right_scale: float,
                 norm_outputs: bool = False):
        super().__init__()
        if norm_outputs:  # constants in front of a norm would do nothing
            if left_scale != right_scale:
                raise ValueError("normed outputs have one scale")
            self.scale = left_scale
            left_scale = right_scale = 1.0
        self.left, self.right = left, right
        for side, scale in ((left, left_scale), (right, right_scale)):
            if scale != 1.0:
                side.scaled(scale)
        self.width, self.norm_outputs = width, norm_outputs
        self._alloc()

    def _alloc(self) -> None:
        wp = pad32(self.width)
        self.inp = _param(self.left.cols + self.right.cols, wp)
        if self.norm_outputs:
            self.outs = nn.ParameterList(
                [_param(wp, m.out_cols) for _, m in self._sides()])
            self.out_norms = nn.ParameterList([_param(wp), _param(wp)])
        else:
            self.o = _param(wp, self.left.out_cols + self.right.out_cols)

    def _sides(self):
        return ("left.", self.left), ("right.", self.right)

    def fit(self, get: Get) -> None:
        """sizes that only a checkpoint's tensors tell"""
        if hasattr(self.right, "fit"):
            self.right.fit(lambda name: get("right." + name))
            self._alloc()

    def shapes(self) -> dict:
        out = {p + k: s for p, m in self._sides()
               for k, s in m.shapes().items()}
        if self.norm_outputs:
            out.update({p + "out": (self.width,) for p, _ in self._sides()})
        return out

    def pack(self, get: Get) -> None:
        row = col = 0
        for i, (p, m) in enumerate(self._sides()):
            def of(name, p=p):
                return get(p + name)

            m.pack_in(self.inp.data[row:row + m.cols], of)
            if self.norm_outputs:
                m.pack_out(self.outs[i].data, of)
                _fill(self.out_norms[i].data, of("out"))
            else:
                m.pack_out(self.o.data[:, col:col + m.out_cols], of)
            m.pack_own(of)
            row += m.cols
            col += m.out_cols

    def finalize(self) -> None:
        self.left.finalize(self.inp.device)
        self.right.finalize()

    def cache_layout(self) -> tuple:
        return "both", self.left.page_layout(), self.right.state_layout()

    def _contexts(self, h, batch, cache, left, right) -> None:
        pages, state = cache
        z = linear(h, self.inp)
        self.left.attend(z[:, :self.left.cols], batch, pages, left)
        self.right.scan(z[:, self.left.cols:], batch, *state, right)

    def forward(self, h, batch, cache, carry):
        n = self.left.out_cols
        ctx = h.new_empty(h.shape[0], self.o.shape[1])
        self._contexts(h, batch, cache, ctx[:, :n], ctx[:, n:])
        return linear(ctx, self.o)

    def branches(self, h, batch, cache
                 ) -> List[Tuple[torch.Tensor, torch.Tensor]]:
        """(output, weight of its norm) of both sides"""
        ctx = [h.new_empty(h.shape[0], m.out_cols) for _, m in self._sides()]
        self._contexts(h, batch, cache, *ctx)
        return [(linear(c, w), norm.data) for c, w, norm in
                zip(ctx, self.outs, self.out_norms)]


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


class DenseMlp(nn.Module):
    """down(xielu(up h)): a z^2 + z / 2 above zero, b (e^z - 1 - z) + z / 2
    below, a = softplus(p) and b = 1/2 + softplus(q) of two learned numbers.
    The layer can take the product with ``down`` along with another."""

    def __init__(self, width: int, ff: int):
        super().__init__()
        self.width, self.ff = width, ff
        w, f = pad32(width), pad32(ff)
        self.out_cols = f
        self.up = _param(f, w)
        self.act = _param(2)
        self._coef: Optional[torch.Tensor] = None  # (a, b) in float

    def shapes(self) -> dict:
        return {"up": (self.ff, self.width), "down": (self.width, self.ff),
                "act": (2,)}

    def pack(self, get: Get) -> None:
        _fill(self.up.data, get("up"))
        _fill(self.act.data, get("act"))

    def pack_out(self, w: torch.Tensor, get: Get) -> None:
        _fill(w, get("down"))

    def finalize(self) -> None:
        a, b = torch.nn.functional.softplus(self.act.data.double())
        self._coef = torch.stack([a, b + 0.5]).float()

    def context(self, h, out) -> None:
        """what ``down`` multiplies, into out [T, out_cols]"""
        lm.xielu(linear(h, self.up), self._coef, out)


class ExpertMlp(nn.Module):
    """Experts down(act(up h)) or, ``gated``, down(act(gate h) * (up h)),
    of which each token takes ``top`` (csrc/lm/moe.hip). The weighted sum is
    left to the kernel that follows: forward -> (rows of all slots,
    (pos, share)); a slot with pos -1 stands for the input itself.

    Default routing: the largest logits, weighed by the softmax over those.
    ``correction``: scores are the softmax over all outputs and weigh the
    chosen experts as they are, the choice adds a learned term; ``groups``
    (count, keep): only the best groups of outputs are chosen from;
    ``identity``: so many more outputs stand for the input. ``shared_ff``: an
    expert of that size for every token, times the sigmoid of a projection;
    it is held as one or more slices of the experts' size, whose outputs add
    up."""

    def __init__(self, width: int, ff: int, experts: int, top: int,
                 act: str = "relu2", gated: bool = False,
                 correction: bool = False,
                 groups: Optional[Tuple[int, int]] = None, identity: int = 0,
                 shared_ff: Optional[int] = None):
        super().__init__()
        outputs = experts + identity
        if not 1 <= top <= outputs:
            raise ValueError("{} of {} experts".format(top, outputs))
        count, keep = groups or (1, 1)
        if not 1 <= keep <= count or outputs % count:
            raise ValueError("best {} of {} groups of {} experts".format(
                keep, count, outputs))
        if keep * (outputs // count) < top:
            raise ValueError("{} experts from {} groups of {}".format(
                top, keep, outputs // count))
        if gated and act != "silu":
            raise ValueError("no gated experts with '{}'".format(act))
        if not correction and (groups or identity):
            raise ValueError("groups and identity experts go with scores "
                             "over all outputs")
        self.width, self.ff, self.shared_ff = width, ff, shared_ff
        self.act = "swiglu" if gated else act
        self.experts, self.top, self.identity = experts, top, identity
        w, f = pad32(width), pad32(ff)
        self.n_shared = 0 if shared_ff is None else -(-shared_ff // f)
        self.how = lm.Routing(top, correction, count, keep, identity,
                              self.n_shared)
        self.gated = gated
        self.router = _param(outputs + (1 if self.n_shared else 0), w)
        self.correction = _param(outputs) if correction else None
        self._correction = None  # in float, whatever the products' type
        n = experts + self.n_shared
        self.up = _param(n, (2 if gated else 1) * f, w)
        self.down = _param(n, w, f)

    @property
    def has_skip(self) -> bool:
        return self.identity > 0

    def shapes(self) -> dict:
        out = {"router": (self.experts + self.identity, self.width)}
        if self.correction is not None:
            out["correction"] = (self.experts + self.identity,)

        def expert(p, ff):
            for k in ("gate", "up") if self.gated else ("up",):
                out[p + k] = (ff, self.width)
            out[p + "down"] = (self.width, ff)

        for e in range(self.experts):
            expert("e{}.".format(e), self.ff)
        if self.n_shared:
            expert("shared.", self.shared_ff)
            out["shared.sg"] = (1, self.width)
        return out

    def _pack_expert(self, e: int, up, gate, down) -> None:
        if self.gated:  # rows in pairs
            pairs = self.up.data[e].view(-1, 2, self.up.shape[2])
            _fill(pairs[:, 0], gate)
            _fill(pairs[:, 1], up)
        else:
            _fill(self.up.data[e], up)
        _fill(self.down.data[e], down)

    def pack(self, get: Get) -> None:
        _fill(self.router.data, get("router"))
        if self.correction is not None:
            _fill(self.correction.data, get("correction"))

        def expert(p):
            return (get(p + "up"), get(p + "gate") if self.gated else None,
                    get(p + "down"))

        for e in range(self.experts):
            self._pack_expert(e, *expert("e{}.".format(e)))
        if self.n_shared:
            _fill(self.router.data[self.experts + self.identity:],
                  get("shared.sg"))
            up, gate, down = expert("shared.")
            f = self.down.shape[2]
            for i in range(self.n_shared):
                part = slice(i * f, (i + 1) * f)
                self._pack_expert(
                    self.experts + i, up[part],
                    gate[part] if self.gated else None, down[:, part])

    def finalize(self) -> None:
        if self.correction is not None:
            self._correction = self.correction.data.float()

    def forward(self, h):
        rows = lm.expert_tile_rows(
            h.shape[0], self.experts, self.top, h.dtype,
            (self.up.shape[2], self.down.shape[2]))
        plan = lm.moe_route(h, self.router, self.how, rows, self._correction)
        hidden = lm.moe_gemm(h, self.up, plan, self.act, gather=True)
        out = lm.moe_gemm(hidden, self.down, plan, "none", gather=False)
        return out, (plan.pos, plan.share)
