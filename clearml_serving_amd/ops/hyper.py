"""Hyper-connections: a residual of several float streams per token
(csrc/lm/hyper.hip), and the cap on logits. GPU tensors run the kernels, CPU
tensors the equations in PyTorch."""

from typing import Optional, Tuple

import torch

from . import require_lm_ext
from .lm import _rms_inv

MAX_STREAMS = 8


def entry_coef(w_in: torch.Tensor, gain: torch.Tensor) -> torch.Tensor:
    """what ``embed`` needs: in [S], gain of the norm"""
    return torch.cat([w_in.float(), gain.float().view(1)])


def step_coef(mix: torch.Tensor, out: torch.Tensor, mult: float,
              w_in: torch.Tensor, gain: torch.Tensor) -> torch.Tensor:
    """what ``step`` needs: a sublayer's mix [from, to] and out times
    ``mult``, and the next sublayer's in and gain"""
    return torch.cat([mix.float().reshape(-1), mult * out.float(),
                      w_in.float(), gain.float().view(1)])


def _norm(u, gain, n, eps, dtype):
    return (u * _rms_inv(u, n, eps) * gain).to(dtype)


def embed(tokens: torch.Tensor, table: torch.Tensor, coef: torch.Tensor,
          streams: int, n: int, eps: float
          ) -> Tuple[torch.Tensor, torch.Tensor]:
    """-> (x float [T, streams, width], all the embedding; h = norm of the
    first sublayer's sum of them, in the table's type). n: true width"""
    if table.is_cuda:
        x, h = require_lm_ext("hyper_embed").lm_hyper_embed(
            tokens, table, coef, streams, n, eps)
        return x, h
    rows = table[tokens.clamp(0, table.shape[0] - 1)].float()
    x = rows[:, None].repeat(1, streams, 1)
    u = (x * coef[:streams, None]).sum(1)
    return x, _norm(u, coef[streams], n, eps, table.dtype)


def step(o: torch.Tensor, x: torch.Tensor, coef: torch.Tensor, n: int,
         eps: float, last: bool = False,
         mix: Optional[Tuple[torch.Tensor, torch.Tensor]] = None,
         skip: Optional[torch.Tensor] = None) -> torch.Tensor:
    """A sublayer's output y goes back into the streams x, in place; -> the
    next sublayer's normed input, in o's type. y = o [T, width], or with
    ``mix`` (pos, share) [T, slots] the sum of share * o[pos], where a slot
    without a row (pos < 0) stands for skip[t]. ``last``: the streams are not
    needed again and not written."""
    if o.is_cuda:
        pos, share = mix if mix is not None else (None, None)
        return require_lm_ext("hyper_step").lm_hyper_step(
            o, x, coef, n, eps, last, pos, share, skip)
    s = x.shape[1]
    y = o.float()
    if mix is not None:
        pos, share = mix
        rows = y[pos.long().clamp(min=0)]
        if skip is not None:
            rows = torch.where((pos < 0)[..., None],
                               skip.float()[:, None], rows)
        y = (rows * share[..., None]).sum(1)
    a, b, w_in = coef[:s * s].view(s, s), coef[s * s:s * s + s], \
        coef[s * s + s:s * s + 2 * s]
    new = (torch.einsum("tsw,sd->tdw", x, a)
           + b[None, :, None] * y[:, None])
    if not last:
        x.copy_(new)
    return _norm((new * w_in[:, None]).sum(1), coef[-1], n, eps, o.dtype)


def soft_cap(z: torch.Tensor, n: int, cap: float) -> torch.Tensor:
    """cap * tanh(z / cap) of the first n columns, in float"""
    if z.is_cuda:
        return require_lm_ext("soft_cap").lm_soft_cap(z, n, cap)
    return cap * torch.tanh(z[:, :n].float() / cap)
