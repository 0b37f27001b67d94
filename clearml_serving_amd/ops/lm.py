"""Token-batch ops: latent attention, gated linear recurrence and the norms
around them, on one flat batch of tokens from many sequences.

GPU tensors run the kernels in ``csrc/lm`` (bf16, or float for exact 32-bit
runs) and need ``_hip_lm.so``; CPU tensors run the equations in PyTorch.

Operands are padded: ``pad32`` of every feature size, zeros behind the true
size, which leaves every product and sum of squares unchanged.
"""

from typing import Optional, Tuple

import torch

from . import require_lm_ext


def pad32(n: int) -> int:
    return (n + 31) // 32 * 32


# --------------------------------------------------------------------- #
# residual stream
# --------------------------------------------------------------------- #
def embed_stream(tokens: torch.Tensor, table: torch.Tensor
                 ) -> Tuple[torch.Tensor, torch.Tensor]:
    """-> (x float [T, width], h = x in the table's type)"""
    if table.is_cuda:
        x, h = require_lm_ext("embed").lm_embed(tokens, table)
        return x, h
    x = table[tokens.clamp(0, table.shape[0] - 1)].float()
    return x, x.to(table.dtype)


def _rms_inv(v: torch.Tensor, n: int, eps: float) -> torch.Tensor:
    return (v.pow(2).sum(-1, keepdim=True) / n + eps).rsqrt()


def post_norm_add(o: torch.Tensor, bias: Optional[torch.Tensor],
                  weight: torch.Tensor, x: torch.Tensor, n: int,
                  eps: float) -> torch.Tensor:
    """x += v / rms(v) * (1 + weight), v = o + bias, in place on the float
    stream; returns x in o's type. ``n``: true row size."""
    if o.is_cuda:
        return require_lm_ext("post_norm_add").lm_post_norm_add(
            o, bias, weight, x, n, eps)
    v = o.float()
    if bias is not None:
        v = v + bias.float()
    x += v * _rms_inv(v, n, eps) * (1.0 + weight.float())
    return x.to(o.dtype)


def output_norm(x: torch.Tensor, rows: Optional[torch.Tensor],
                weight: torch.Tensor, n: int, eps: float,
                scale: float = 1.0) -> torch.Tensor:
    """x[rows] / rms * (1 + weight) * scale in the weight's type."""
    if x.is_cuda:
        return require_lm_ext("output_norm").lm_output_norm(
            x, rows, weight, n, eps, scale)
    v = x if rows is None else x[rows.long()]
    return (v * _rms_inv(v, n, eps) * (1.0 + weight.float()) * scale
            ).to(weight.dtype)


def gelu_mul(gate_up: torch.Tensor, bias: Optional[torch.Tensor]
             ) -> torch.Tensor:
    """gelu_tanh(gate + bg) * (up + bu); gate_up = [gate | up] columns."""
    if gate_up.is_cuda:
        return require_lm_ext("gelu_mul").lm_gelu_mul(gate_up, bias)
    v = gate_up.float()
    if bias is not None:
        v = v + bias.float()
    g, u = v.chunk(2, dim=-1)
    return (torch.nn.functional.gelu(g, approximate="tanh") * u
            ).to(gate_up.dtype)


def gather_rows(src: torch.Tensor, idx: torch.Tensor) -> torch.Tensor:
    """rows of ``src`` (last dim kept, the others flattened)"""
    if src.is_cuda:
        return require_lm_ext("gather_rows").lm_gather_rows(src, idx)
    return src.reshape(-1, src.shape[-1])[idx.long()]


# --------------------------------------------------------------------- #
# latent attention
# --------------------------------------------------------------------- #
def _rotate_pairs_(v: torch.Tensor, positions: torch.Tensor,
                   inv_freq: torch.Tensor) -> None:
    """v [T, ..., >= 2 * pairs]: neighbours (2i, 2i+1), in place"""
    n = 2 * inv_freq.numel()
    ang = positions.float()[:, None] * inv_freq[None, :]
    while ang.dim() < v.dim():
        ang = ang.unsqueeze(1)
    c, s = ang.cos(), ang.sin()
    a, b = v[..., 0:n:2].float(), v[..., 1:n:2].float()
    a, b = a * c - b * s, b * c + a * s
    v[..., 0:n:2] = a.to(v.dtype)
    v[..., 1:n:2] = b.to(v.dtype)


def latent_prep(qkv: torch.Tensor, positions: torch.Tensor,
                slot_mapping: torch.Tensor, inv_freq: torch.Tensor,
                heads: int, dp: int, rp: int, cp: int, kv_rank: int,
                eps: float, kv_norm: Optional[torch.Tensor],
                cache: Optional[torch.Tensor],
                q_abs: Optional[torch.Tensor]) -> None:
    """Rotate q; with ``kv_norm`` (the layer owns its latent) also normalise
    c, rotate the shared key part and write the cache row of each token.

    qkv rows are [heads x (dp | rp)] and, if owned, [cp | rp] behind them.
    The rotated part of the first len(q_abs) tokens goes into
    q_abs [n, heads, cp + rp] (absorbed attention), that of the others stays
    in place."""
    n_abs = 0 if q_abs is None else q_abs.shape[0]
    if qkv.is_cuda:
        require_lm_ext("latent_prep").lm_latent_prep(
            qkv, positions, slot_mapping, inv_freq, heads, dp, rp, cp,
            kv_rank, eps, kv_norm, cache, q_abs, n_abs)
        return
    t = qkv.shape[0]
    q = qkv[:, :heads * (dp + rp)].view(t, heads, dp + rp)
    _rotate_pairs_(q[..., dp:], positions, inv_freq)
    if n_abs:
        q_abs[..., cp:] = q[:n_abs, :, dp:]
    if kv_norm is None:
        return
    lat = qkv[:, heads * (dp + rp):].clone()
    c = lat[:, :cp].float()
    lat[:, :cp] = (c * _rms_inv(c, kv_rank, eps) * kv_norm.float()
                   ).to(lat.dtype)
    _rotate_pairs_(lat[:, cp:], positions, inv_freq)
    keep = slot_mapping >= 0
    cache.view(-1, cp + rp)[slot_mapping[keep].long()] = lat[keep]


def head_gemm(a: torch.Tensor, w: torch.Tensor, out: torch.Tensor) -> None:
    """out[t, h] = w[h] @ a[t, h]; w [H, N, K], strided a and out."""
    if a.is_cuda:
        require_lm_ext("head_gemm").lm_head_gemm(a, w, out)
        return
    out.copy_(torch.matmul(a.transpose(0, 1).float(),
                           w.float().transpose(1, 2)).transpose(0, 1))


def _sink_softmax(s: torch.Tensor, sink: torch.Tensor) -> torch.Tensor:
    """softmax over the last dim with exp(sink) added to the denominator"""
    full = torch.cat([s, sink.expand(*s.shape[:-1], 1)], dim=-1)
    return torch.softmax(full, dim=-1)[..., :-1]


def latent_attention(q_abs: torch.Tensor, cache: torch.Tensor,
                     block_table: torch.Tensor, tok_seq: torch.Tensor,
                     positions: torch.Tensor, sink: torch.Tensor,
                     scale: float, window: int, cp: int,
                     max_keys: int) -> torch.Tensor:
    """Absorbed form. q_abs [n, H, cp + rp]; each token attends to the cached
    rows of its own sequence up to its position, the last ``window`` of them
    (0: all). ``max_keys``: bound on positions + 1, sizes the launch.
    -> latent sums [n, H, cp]"""
    if q_abs.is_cuda:
        return require_lm_ext("latent_attention").lm_latent_attention(
            q_abs, cache, block_table, tok_seq, positions, sink, scale,
            window, cp, max_keys)
    bs = cache.shape[1]
    rows = cache.view(-1, cache.shape[2])
    out = torch.empty(*q_abs.shape[:2], cp, dtype=q_abs.dtype)
    for t in range(q_abs.shape[0]):
        p = int(positions[t])
        key = torch.arange(max(0, p - window + 1) if window else 0, p + 1)
        blk = block_table[int(tok_seq[t])].long()[key // bs]
        k = rows[blk * bs + key % bs].float()
        s = (q_abs[t].float() @ k.T) * scale
        w = _sink_softmax(s, sink.float()[:, None])
        out[t] = (w @ k[:, :cp]).to(out.dtype)
    return out


PROMPT_TILE = 128     # queries per workgroup of latent_prompt
PROMPT_MAX_HEAD = 256  # largest padded key and value size it takes


def latent_prompt(q: torch.Tensor, kv: torch.Tensor, lat: torch.Tensor,
                  sink: torch.Tensor, qtiles: torch.Tensor,
                  out: torch.Tensor, heads: int, dp: int, rp: int, cp: int,
                  vp: int, window: int, scale: float) -> None:
    """Expanded form, for prompt portions. q [T, heads * (dp + rp)]; kv
    [rows, heads * dp | heads * vp] keys and values of the gathered cache
    rows lat [rows, cp + rp]; qtiles [n, 6]: first token, tokens, first
    position, first gathered row, its position, gathered rows of the
    sequence. Writes out [T, heads, vp] at the tiles' tokens."""
    if q.is_cuda:
        require_lm_ext("latent_prompt").lm_latent_prompt(
            q, kv, lat, sink, qtiles, out, heads, dp, rp, cp, vp, window,
            scale)
        return
    for t0, n, p0, r0, k_lo, nk in qtiles.tolist():
        qq = q[t0:t0 + n, :heads * (dp + rp)].float().view(n, heads, -1)
        rows = kv[r0:r0 + nk].float()
        k = rows[:, :heads * dp].view(nk, heads, dp)
        v = rows[:, heads * dp:].view(nk, heads, vp)
        s = torch.einsum("nhd,khd->hnk", qq[..., :dp], k) + torch.einsum(
            "nhd,kd->hnk", qq[..., dp:], lat[r0:r0 + nk, cp:].float())
        dist = (p0 + torch.arange(n))[:, None] - (k_lo + torch.arange(nk))
        ok = (dist >= 0) & ((dist < window) if window else True)
        w = _sink_softmax((s * scale).masked_fill(~ok, float("-inf")),
                          sink.float()[:, None, None])
        out[t0:t0 + n] = torch.einsum("hnk,khd->nhd", w, v).to(out.dtype)


# --------------------------------------------------------------------- #
# gated linear recurrence
# --------------------------------------------------------------------- #
class RglruWeights:
    """One layer's operands: yx bias [2W], conv taps [taps, W] and bias,
    block-diagonal gates [blocks, k, k] with biases [W], lam [W]."""

    __slots__ = ("byx", "cw", "cb", "ra", "ba", "ri", "bi", "lam")

    def __init__(self, byx, cw, cb, ra, ba, ri, bi, lam):
        self.byx, self.cw, self.cb = byx, cw, cb
        self.ra, self.ba, self.ri, self.bi, self.lam = ra, ba, ri, bi, lam

    def all(self):
        return (self.byx, self.cw, self.cb, self.ra, self.ba, self.ri,
                self.bi, self.lam)


def _rglru_token(yx, w: RglruWeights, state, ring, pos: int, slot: int):
    """one token of one sequence; state/ring rows updated in place"""
    width, taps = w.lam.numel(), w.cw.shape[0]
    y = yx[:width].float() + w.byx[:width].float()
    raw = yx[width:]
    u = w.cb.float() + (raw.float() + w.byx[width:].float()) \
        * w.cw[taps - 1].float()
    live = 0 <= slot < state.shape[0]
    for d in range(1, min(taps - 1, pos) + 1 if live else 1):
        u = u + (ring[slot, (pos - d) % taps].float()
                 + w.byx[width:].float()) * w.cw[taps - 1 - d].float()
    u = u.to(yx.dtype).float()
    ub = u.view(w.ra.shape[0], 1, -1)
    r = torch.sigmoid(torch.matmul(ub, w.ra.float().transpose(1, 2))
                      .view(-1) + w.ba.float())
    i = torch.sigmoid(torch.matmul(ub, w.ri.float().transpose(1, 2))
                      .view(-1) + w.bi.float())
    log_a = -8.0 * r * torch.nn.functional.softplus(w.lam.float())
    s = torch.sqrt(-torch.expm1(2.0 * log_a)) * i * u
    if live:
        if pos > 0:
            s = s + torch.exp(log_a) * state[slot]
        state[slot] = s
        ring[slot, pos % taps] = raw
    return (s * torch.nn.functional.gelu(y, approximate="tanh")).to(yx.dtype)


def rglru_step(yx: torch.Tensor, w: RglruWeights, state: torch.Tensor,
               ring: torch.Tensor, positions: torch.Tensor,
               slots: torch.Tensor, out: torch.Tensor, n: int) -> None:
    """Rows [0, n) of yx [T, 2W] = [y | x]: one token each of n different
    sequences. state [slots, W] float, ring [slots, taps, W]."""
    if n == 0:
        return
    if yx.is_cuda:
        require_lm_ext("rglru_step").lm_rglru_step(
            yx, *w.all(), state, ring, positions, slots, out, n)
        return
    for t in range(n):
        out[t] = _rglru_token(yx[t], w, state, ring, int(positions[t]),
                              int(slots[t]))


def rglru_prefill(yx: torch.Tensor, w: RglruWeights, state: torch.Tensor,
                  ring: torch.Tensor, tiles: torch.Tensor,
                  seqs: torch.Tensor, out: torch.Tensor, tile: int) -> None:
    """Portions of several tokens. tiles [n, 5]: first token, tokens, first
    position, state slot, distance to the portion's start; seqs [m, 6]:
    first tile, tiles, first token, tokens, first position, state slot."""
    if seqs.shape[0] == 0:
        return
    if yx.is_cuda:
        require_lm_ext("rglru_prefill").lm_rglru_prefill(
            yx, *w.all(), state, ring, tiles, seqs, out, tile)
        return
    for _, _, t0, n, p0, slot in seqs.tolist():
        for j in range(n):
            out[t0 + j] = _rglru_token(yx[t0 + j], w, state, ring, p0 + j,
                                       slot)
