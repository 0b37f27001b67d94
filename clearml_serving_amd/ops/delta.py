"""Generalised delta rule on a flat token batch (csrc/lm/delta.hip): GPU
tensors run the kernel, CPU tensors the equations in PyTorch."""

import math
from typing import NamedTuple, Tuple

import torch

from . import require_lm_ext

HEAD_SIZES = (32, 64, 96, 128, 192, 256)  # padded, that the kernel takes


def head_pad(dim: int) -> int:
    for n in HEAD_SIZES:
        if dim <= n:
            return n
    raise ValueError("delta rule: head of {} channels, at most {}".format(
        dim, HEAD_SIZES[-1]))


def chunk_tiles(tiles: int, seqs: int, heads: int) -> int:
    """how many tiles make a chunk of a portion, 0: portions stay whole.
    Chunks are walked twice, and once more without outputs, so cutting pays
    where whole portions leave CUs idle."""
    if seqs == 0 or seqs * heads > 160 or tiles < 6 * seqs:
        return 0
    return max(3, -(-tiles * heads // 1024))


class DeltaWeights(NamedTuple):
    """w2 [heads * dp, rank] and w0 make the decay, ab the removal rate, norm
    weighs the output; [heads * dp] each."""

    w2: torch.Tensor
    w0: torch.Tensor
    ab: torch.Tensor
    norm: torch.Tensor


def delta_rule(z: torch.Tensor, at: Tuple[int, ...], w: DeltaWeights,
               state: torch.Tensor, positions: torch.Tensor,
               slots: torch.Tensor, seqs: torch.Tensor, out: torch.Tensor,
               n_single: int, dim: int, eps: float, out_scale: float,
               n_tiles: int, tile: int) -> None:
    """z [T, cols]: columns ``at`` of r, k, v, g, a (heads * dp each) and of
    the decay's low-rank input. The first n_single tokens are one token each
    of different sequences (``positions``, state ``slots``), the others
    portions: seqs [m, 6] as in ops.lm.rglru_prefill, n_tiles tiles of
    ``tile`` tokens in all. state float [slots, heads, dp, dp] as
    [value][key]; position 0 starts from zero. -> out [T, heads * dp]"""
    if z.is_cuda:
        require_lm_ext("delta_rule").lm_delta_rule(
            z, list(at), w.w2, w.w0, w.ab, w.norm, state, positions, slots,
            seqs, out, n_single, dim, eps, out_scale, n_tiles, tile,
            chunk_tiles(n_tiles, seqs.shape[0], state.shape[1]))
        return
    heads, dp = state.shape[1:3]
    f = z.float()
    r, k, v, g, a = (f[:, c:c + heads * dp].view(-1, heads, dp)
                     for c in at[:5])
    low = torch.tanh(f[:, at[5]:at[5] + w.w2.shape[1]])
    decay = torch.exp(-math.exp(-0.5) * torch.sigmoid(
        low @ w.w2.float().t() + w.w0.float())).view(-1, heads, dp)
    u = k / torch.sqrt(k.pow(2).sum(-1, keepdim=True) + 1e-6)
    b = torch.sigmoid(a + w.ab.float().view(heads, dp)) * u
    todo = [(i, 1, int(positions[i]), int(slots[i]))
            for i in range(n_single)]
    todo += [tuple(s[2:]) for s in seqs.tolist()]
    for t0, n, p0, slot in todo:
        live = 0 <= slot < state.shape[0]
        s = state[slot].clone() if live and p0 > 0 else \
            torch.zeros(heads, dp, dp)
        for t in range(t0, t0 + n):
            x = torch.einsum("hvk,hk->hv", s, u[t])
            s = (s * decay[t][:, None] - x[..., None] * b[t][:, None]
                 + v[t][..., None] * k[t][:, None])
            o = torch.einsum("hvk,hk->hv", s, r[t])
            o = o * (o.pow(2).sum(-1, keepdim=True) / dim + eps).rsqrt()
            out[t] = (out_scale * o.reshape(-1) * w.norm.float()
                      * torch.sigmoid(g[t].reshape(-1))).to(out.dtype)
        if live:
            state[slot] = s
