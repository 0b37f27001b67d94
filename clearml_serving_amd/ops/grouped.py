"""Grouped-query attention on paged rows of a flat token batch
(csrc/lm/gqa.hip, prompt_attn.hip). GPU tensors run the kernels, CPU tensors
the equations in PyTorch.

Cache row: a slice [key kd | value vd] per key/value head. Where the values are
the keys before their norm (``same``), a slice is that projection alone and
behind the slices stands a float per head, the factor of the key's norm; the
norm's weights are part of the query.

Pooled layers also see one row for every block of ``pool`` tokens that lies
wholly in front of the window, the mean of the block's rows. A page holds its
tokens' rows and, behind them, the means of the blocks whose last token it
holds, so pooled rows are allocated and freed with the tokens'.
"""

from typing import NamedTuple, Optional

import torch

from . import require_lm_ext
from .lm import Rotary, _sink_softmax, pad32


class GroupedSpec(NamedTuple):
    """Sizes (padded ``kd``, ``vd``; true ``dim``) and constants of a layer.
    ``window`` 0: all earlier tokens, else also the first ``keep`` tokens, or
    with ``pool`` the means of the blocks of so many tokens in front of it.
    ``cap`` 0: none. ``out_scale`` multiplies the result. ``whole``: norms of
    queries and keys run over all heads at once."""

    heads: int
    kv_heads: int
    kd: int
    vd: int
    dim: int
    same: bool
    window: int
    keep: int
    scale: float
    cap: float
    out_scale: float
    pool: int = 0
    whole: bool = False

    @property
    def slice(self) -> int:
        return self.kd if self.same else self.kd + self.vd

    @property
    def row(self) -> int:
        """cached elements per token"""
        n = self.kv_heads * self.slice
        # a float is two elements of a 16-bit cache
        return n + pad32(2 * self.kv_heads) if self.same else n


def page_rows(block_size: int, pool: int) -> int:
    """rows of a page of ``block_size`` tokens"""
    return block_size + (-(-block_size // pool) if pool else 0)


def page_tokens(rows: int, pool: int) -> int:
    """tokens of a page of ``rows`` rows"""
    return rows * pool // (pool + 1) if pool else rows


def token_row(block, offset, block_size: int, pool: int):
    """row of a token at ``offset`` of page ``block``"""
    return block * page_rows(block_size, pool) + offset


def pooled_row(block, offset, block_size: int, pool: int):
    """row of the mean of the block whose last token is at ``offset`` of page
    ``block``"""
    return (block * page_rows(block_size, pool) + block_size
            + offset // pool)


def _norm_factor(v: torch.Tensor, n: int, eps: float) -> torch.Tensor:
    return (v.float().pow(2).sum(-1, keepdim=True) / n + eps).rsqrt()


def _key_factors(rows: torch.Tensor, s: GroupedSpec) -> torch.Tensor:
    """the floats behind the slices, a view [rows, kv_heads]"""
    at = s.kv_heads * s.slice
    return rows[:, at:].view(torch.float32)[:, :s.kv_heads]


def prepare(z: torch.Tensor, k_at: int, v_at: int, positions: torch.Tensor,
            slot_mapping: torch.Tensor, rot: Optional[Rotary],
            s: GroupedSpec, q_norm: Optional[torch.Tensor],
            k_norm: Optional[torch.Tensor], eps: float,
            first: Optional[torch.Tensor], lam: float,
            cache: torch.Tensor, bias: Optional[torch.Tensor] = None
            ) -> None:
    """z [T, cols]: queries at column 0, keys at k_at, values at v_at; ``bias``
    [cols] is added first. Norms (per head, weights [kd], or over all heads,
    weights [heads * kd]) and rotates queries in place and keys on their way to
    the cache rows of ``slot_mapping`` (page * tokens of a page + offset);
    ``first`` [T, kv_heads * vd]: values become (1 - lam) v + lam first."""
    if z.is_cuda:
        require_lm_ext("grouped_prep").lm_grouped_prep(
            z, k_at, -1 if s.same else v_at, positions, slot_mapping,
            None if rot is None else rot.inv_freq,
            1.0 if rot is None else rot.gain, s.heads, s.kv_heads, s.kd,
            s.vd, s.dim, q_norm, k_norm, eps, first, lam, cache, bias,
            s.whole, s.pool)
        return
    t, g = z.shape[0], s.kv_heads
    if bias is not None:
        z.copy_(z.float() + bias.float())
    q = z[:, :s.heads * s.kd].view(t, s.heads, s.kd)
    k = z[:, k_at:k_at + g * s.kd].reshape(t, g, s.kd)
    qf, kf = q.float(), k.float()
    if s.whole:
        qf = (qf.view(t, -1) * _norm_factor(q.reshape(t, -1), s.heads * s.dim,
                                            eps) * q_norm.float()).view_as(q)
        kf = (kf.view(t, -1) * _norm_factor(k.reshape(t, -1), g * s.dim, eps)
              * k_norm.float()).view_as(k)
        q_norm = k_norm = None
    if q_norm is not None:
        qf = qf * _norm_factor(q, s.dim, eps) * q_norm.float()
    keep = slot_mapping >= 0
    at = slot_mapping[keep].long()
    bs = page_tokens(cache.shape[1], s.pool)
    at = token_row(at // bs, at % bs, bs, s.pool)
    rows = cache.view(-1, cache.shape[-1])
    if s.same:
        new = rows[at]  # a copy
        new[:, :g * s.kd] = k.reshape(t, -1)[keep]
        _key_factors(new, s)[:] = 1.0
        if k_norm is not None:
            qf = qf * k_norm.float()
            _key_factors(new, s)[:] = _norm_factor(k, s.dim, eps)[keep, :, 0]
        rows[at] = new
    else:
        if k_norm is not None:
            kf = kf * _norm_factor(k, s.dim, eps) * k_norm.float()
        v = z[:, v_at:v_at + g * s.vd].reshape(t, g, s.vd)
        if first is not None:
            v = ((1.0 - lam) * v.float()
                 + lam * first.reshape(t, g, s.vd).float())
        if rot is not None:
            kf = kf.clone()
            rot.rotate_(kf, positions)
        new = torch.cat([kf.to(z.dtype), v.to(z.dtype)], -1).view(t, -1)
        rows[at] = new[keep]
    if rot is not None:
        qf = qf.clone()
        rot.rotate_(qf, positions)
    q.copy_(qf)


def pool_rows(cache: torch.Tensor, block_table: torch.Tensor,
              tok_seq: torch.Tensor, positions: torch.Tensor,
              pool: int) -> None:
    """Writes the mean row of every block of ``pool`` tokens that one of the
    given tokens ends; the block's rows are in the cache."""
    if cache.is_cuda:
        require_lm_ext("grouped_pool").lm_grouped_pool(
            cache, block_table, tok_seq, positions, pool)
        return
    bs = page_tokens(cache.shape[1], pool)
    rows = cache.view(-1, cache.shape[2])
    for t, p in enumerate(positions.tolist()):
        if (p + 1) % pool:
            continue
        pages = block_table[int(tok_seq[t])].long()
        key = torch.arange(p + 1 - pool, p + 1)
        mean = rows[token_row(pages[key // bs], key % bs, bs, pool)].float()
        rows[pooled_row(pages[p // bs], p % bs, bs, pool)] = \
            mean.mean(0).to(cache.dtype)


def _attend(q, rows, see, sink, s: GroupedSpec):
    """q [n, H * kd], cache rows [k, row], see [n, k] -> [n, H * vd]"""
    n, per = q.shape[0], s.heads // s.kv_heads
    slices = rows[:, :s.kv_heads * s.slice].view(-1, s.kv_heads, s.slice)
    k = slices[..., :s.kd].float().repeat_interleave(per, 1)
    v = (slices if s.same else slices[..., s.kd:]).float() \
        .repeat_interleave(per, 1)
    sc = torch.einsum("nhd,khd->hnk", q.float().view(n, s.heads, s.kd), k)
    if s.same:
        sc = sc * _key_factors(rows, s).repeat_interleave(per, 1).t()[:, None]
    sc = sc * s.scale
    if s.cap:
        sc = s.cap * torch.tanh(sc / s.cap)
    w = _sink_softmax(sc.masked_fill(~see, float("-inf")),
                      None if sink is None else sink.float()[:, None, None])
    return s.out_scale * torch.einsum("hnk,khd->nhd", w, v).reshape(n, -1)


def _sees(qpos, kpos, s: GroupedSpec):
    d = qpos[:, None] - kpos[None, :]
    see = d >= 0
    if s.window:
        see = see & ((d < s.window) | (kpos[None, :] < s.keep))
    return see


def attention(q: torch.Tensor, cache: torch.Tensor, block_table: torch.Tensor,
              tok_seq: torch.Tensor, positions: torch.Tensor,
              sink: Optional[torch.Tensor], out: torch.Tensor, n: int,
              s: GroupedSpec, max_keys: int) -> None:
    """The first n tokens of q [T, H * kd], each on its own sequence's cache
    rows, into out [T, H * vd]. ``sink`` [H] or None. ``max_keys``: bound on
    positions + 1, sizes the launch."""
    if q.is_cuda:
        require_lm_ext("grouped_attention").lm_grouped_attention(
            q, cache, block_table, tok_seq, positions, sink, out, n, s.heads,
            s.kv_heads, s.kd, s.vd, s.same, s.window, s.keep, s.pool, s.scale,
            s.cap, s.out_scale, max_keys)
        return
    bs = page_tokens(cache.shape[1], s.pool)
    rows = cache.view(-1, cache.shape[2])
    for t in range(n):
        p = int(positions[t])
        key = torch.arange(p + 1)
        key = key[_sees(torch.tensor([p]), key, s)[0]]
        pages = block_table[int(tok_seq[t])].long()
        at = token_row(pages[key // bs], key % bs, bs, s.pool)
        if s.pool:
            blocks = max(0, p + 1 - s.window) // s.pool
            last = torch.arange(blocks) * s.pool + s.pool - 1
            at = torch.cat([pooled_row(pages[last // bs], last % bs, bs,
                                       s.pool), at])
        got = _attend(q[t:t + 1], rows[at],
                      torch.ones(1, len(at), dtype=torch.bool), sink, s)
        out[t] = got[0].to(out.dtype)


def prompt(q: torch.Tensor, rows: torch.Tensor, sink: Optional[torch.Tensor],
           qtiles: torch.Tensor, out: torch.Tensor, s: GroupedSpec) -> None:
    """Prompt portions on gathered cache rows [n, row]; qtiles [n, 6]: first
    token, tokens, first position, first gathered row, what the number of a
    row behind the ``keep`` first lacks to its position, gathered rows of the
    sequence. With ``pool`` a seventh column: pooled rows, which come first,
    as ``keep`` ones do. Writes out [T, H * vd] at the tiles' tokens."""
    if q.is_cuda:
        require_lm_ext("grouped_prompt").lm_grouped_prompt(
            q, rows, sink, qtiles, out, s.heads, s.kv_heads, s.kd, s.vd,
            s.same, s.window, s.keep, s.pool, s.scale, s.cap, s.out_scale)
        return
    for t0, n, p0, r0, skip, nk, *pooled in qtiles.tolist():
        qpos = p0 + torch.arange(n)
        kpos = torch.arange(nk)
        if s.pool:
            kpos, blocks = kpos[pooled[0]:] + skip, kpos[:pooled[0]]
            last = blocks * s.pool + s.pool - 1
            see = torch.cat([last[None] <= qpos[:, None] - s.window,
                             _sees(qpos, kpos, s)], 1)
        else:
            kpos[s.keep:] += skip
            see = _sees(qpos, kpos, s)
        out[t0:t0 + n] = _attend(q[t0:t0 + n], rows[r0:r0 + nk], see, sink,
                                 s).to(out.dtype)
