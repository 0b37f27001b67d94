"""Linear recurrences with one decay per head on a flat token batch
(csrc/lm/linear_state.hip): the gated delta rule and the state-space
recurrence. GPU tensors run the kernels, CPU tensors the equations in PyTorch.

A product of the input holds, per token, [q | k | v | gate | a | b]: q and k
``groups`` heads of ``kp`` channels, v and gate ``heads`` of ``vp``, a and b one
number per head (in ``sp`` columns). q, k and v pass a causal convolution over
time and SiLU. Per head, with the q and k of its group:

    g = -exp(a_log) softplus(a + dt_bias)
    delta:   q, k become unit vectors, q times dim^-1/2; b = sigmoid(b)
             S <- e^g S;  u = b (v - S^T k);  S <- S + k u^T;  o = S^T q
             out = o / rms(o) * norm * silu(gate)
    else:    d = softplus(a + dt_bias)
             S <- e^g S + d k v^T;  o = S^T q + skip v
             out = p / rms(p) * norm, p = o * silu(gate), in ``parts`` parts

State float [slots, heads, vp, kp]; the convolution's past inputs are a ring
[slots, taps, channels] indexed by position. Position 0 starts from zero.
"""

from typing import NamedTuple, Optional

import torch

from . import require_lm_ext
from .lm import pad32

KEY_SIZES = (32, 64, 96, 128, 256)  # padded, that the kernels take
MAX_TAPS = 8


def key_pad(dim: int) -> int:
    for n in KEY_SIZES:
        if dim <= n:
            return n
    raise ValueError("recurrence with {} key channels, at most {}".format(
        dim, KEY_SIZES[-1]))


class StateSpec(NamedTuple):
    """Sizes (padded ``kp``, ``vp``; true ``dim``, ``vdim``) and constants."""

    delta: bool
    heads: int
    groups: int
    dim: int
    vdim: int
    taps: int
    parts: int
    eps: float

    @property
    def kp(self) -> int:
        return key_pad(self.dim)

    @property
    def vp(self) -> int:
        return pad32(self.vdim)

    @property
    def sp(self) -> int:
        return pad32(self.heads)

    @property
    def k_at(self) -> int:
        return self.groups * self.kp

    @property
    def v_at(self) -> int:
        return 2 * self.k_at

    @property
    def channels(self) -> int:
        """that the convolution takes"""
        return self.v_at + self.heads * self.vp

    @property
    def a_at(self) -> int:
        return self.channels + self.heads * self.vp

    @property
    def cols(self) -> int:
        return self.a_at + (2 if self.delta else 1) * self.sp

    def layout(self) -> tuple:
        """of a slot: state and ring, as models' cache_layout names them"""
        return ("state", (self.heads, self.vp, self.kp),
                (self.taps, self.channels))


def segment_tiles(tiles: int, seqs: int, s: StateSpec) -> int:
    """how many tiles make a segment of a portion, 0: portions stay whole.
    Segments are walked twice (three times with P), so cutting pays where
    whole portions leave CUs idle."""
    units = seqs * s.heads * -(-s.vp // 64)  # workgroups without segments
    if units == 0 or units > (96 if s.delta else 160) or tiles < 8 * seqs:
        return 0
    parts = max(2, min(tiles // (4 * seqs), 256 // units))
    return -(-tiles // (seqs * parts))


class StateWeights(NamedTuple):
    """conv [taps, channels] and its bias, a_log, dt_bias, skip [heads], norm
    [heads * vp]; skip without ``delta`` only"""

    conv: torch.Tensor
    conv_b: Optional[torch.Tensor]
    a_log: torch.Tensor
    dt_bias: torch.Tensor
    skip: Optional[torch.Tensor]
    norm: torch.Tensor


def _silu(v):
    return v * torch.sigmoid(v)


def _token(z, s: StateSpec, w: StateWeights, state, ring, pos: int,
           slot: int):
    """one token of one sequence: -> o [heads, vp]; state and ring rows
    advance in place"""
    live = 0 <= slot < state.shape[0]
    raw = z[:s.channels]
    x = raw.float() * w.conv[s.taps - 1].float()
    for d in range(1, min(s.taps - 1, pos) + 1 if live else 1):
        x = x + ring[slot, (pos - d) % s.taps].float() \
            * w.conv[s.taps - 1 - d].float()
    if w.conv_b is not None:
        x = x + w.conv_b.float()
    x = _silu(x)
    per = s.heads // s.groups
    q, k = (x[at:at + s.k_at].view(s.groups, s.kp) for at in (0, s.k_at))
    v = x[s.v_at:].view(s.heads, s.vp)
    step = torch.nn.functional.softplus(
        z[s.a_at:s.a_at + s.heads].float() + w.dt_bias.float())
    decay = torch.exp(-torch.exp(w.a_log.float()) * step)
    if s.delta:
        q, k = (y / torch.sqrt(y.pow(2).sum(-1, keepdim=True) + 1e-6)
                for y in (q, k))
        q = q * s.dim ** -0.5
        step = torch.sigmoid(z[s.a_at + s.sp:][:s.heads].float())
    q, k = (y.repeat_interleave(per, 0) for y in (q, k))
    m = torch.zeros(s.heads, s.vp, s.kp) if not live or pos == 0 \
        else state[slot]
    m = m * decay[:, None, None]
    u = v
    if s.delta:
        u = v - torch.einsum("hvk,hk->hv", m, k)
    m = m + (step[:, None] * u)[..., None] * k[:, None]
    o = torch.einsum("hvk,hk->hv", m, q)
    if not s.delta:
        o = o + w.skip.float()[:, None] * v
    if live:
        state[slot] = m
        ring[slot, pos % s.taps] = raw
    return o


def _finish(o, gate, s: StateSpec, w: StateWeights):
    """o, gate [heads, vp] -> [heads * vp]"""
    gate = _silu(gate.float())
    p = o if s.delta else o * gate
    rows = p[:, :s.vdim].reshape(s.heads if s.delta else s.parts, -1)
    rows = rows * (rows.pow(2).mean(-1, keepdim=True) + s.eps).rsqrt()
    p = torch.zeros_like(o)
    p[:, :s.vdim] = rows.view(s.heads, s.vdim)
    p = p * w.norm.float().view(s.heads, s.vp)
    return (p * gate if s.delta else p).view(-1)


def linear_state(z: torch.Tensor, s: StateSpec, w: StateWeights,
                 state: torch.Tensor, ring: torch.Tensor,
                 positions: torch.Tensor, slots: torch.Tensor,
                 tiles: torch.Tensor, seqs: torch.Tensor, tile: int,
                 n_single: int, out: torch.Tensor) -> None:
    """z [T, cols] -> out [T, heads * vp]. The first n_single tokens are one
    token each of different sequences (``positions``, state ``slots``), the
    others portions: tiles of ``tile`` (64) tokens, seqs as in
    ops.lm.rglru_prefill."""
    if z.is_cuda:
        require_lm_ext("linear_state").lm_linear_state(
            z, s.delta, s.heads, s.groups, s.dim, s.vdim, s.parts, s.eps,
            w.conv, w.conv_b, w.a_log, w.dt_bias, w.skip, w.norm, state,
            ring, positions, slots, tiles, seqs, tile,
            segment_tiles(tiles.shape[0], seqs.shape[0], s), n_single, out)
        return
    todo = [(i, 1, int(positions[i]), int(slots[i]))
            for i in range(n_single)]
    todo += [tuple(r[2:]) for r in seqs.tolist()]
    for t0, n, p0, slot in todo:
        for t in range(n):
            row = z[t0 + t]
            o = _token(row, s, w, state, ring, p0 + t, slot)
            out[t0 + t] = _finish(
                o, row[s.channels:s.a_at].view(s.heads, s.vp), s,
                w).to(out.dtype)
