"""Token-batch ops: latent attention, gated linear recurrence, mixture of
experts and the norms around them, on one flat batch of tokens from many
sequences.

GPU tensors run the kernels in ``csrc/lm`` (bf16, or float for exact 32-bit
runs) and need ``_hip_lm.so``; CPU tensors run the equations in PyTorch.

Operands are padded: ``pad32`` of every feature size, zeros behind the true
size, which leaves every product and sum of squares unchanged.
"""

import math
from typing import List, NamedTuple, Optional, Sequence, Tuple, Union

import torch

from . import require_lm_ext


def pad32(n: int) -> int:
    return (n + 31) // 32 * 32


# --------------------------------------------------------------------- #
# residual stream
# --------------------------------------------------------------------- #
class RowNorm:
    """x / rms(x) * (offset + weight) over rows of true size ``n``."""

    __slots__ = ("weight", "n", "eps", "offset")

    def __init__(self, weight: torch.Tensor, n: int, eps: float,
                 offset: float):
        self.weight, self.n, self.eps, self.offset = weight, n, eps, offset

    def __call__(self, v: torch.Tensor) -> torch.Tensor:  # CPU equations
        return v * _rms_inv(v, self.n, self.eps) * (
            self.offset + self.weight.float())


def _rms_inv(v: torch.Tensor, n: int, eps: float) -> torch.Tensor:
    return (v.pow(2).sum(-1, keepdim=True) / n + eps).rsqrt()


def _next_input(x, norm: Optional[RowNorm], dtype, out):
    h = (x if norm is None else norm(x)).to(dtype)
    return h if out is None else out.copy_(h)


def embed_stream(tokens: torch.Tensor, table: torch.Tensor,
                 norm: Optional[RowNorm] = None,
                 out: Optional[torch.Tensor] = None,
                 copy: Optional[torch.Tensor] = None
                 ) -> Tuple[torch.Tensor, torch.Tensor]:
    """-> (x float [T, width], h: x, or norm(x), in the table's type, in
    ``out`` if given). ``copy`` also receives the rows as they are."""
    if table.is_cuda:
        w, n, eps, off = (None, table.shape[1], 0.0, 0.0) if norm is None \
            else (norm.weight, norm.n, norm.eps, norm.offset)
        x, h = require_lm_ext("embed").lm_embed(tokens, table, w, off, n,
                                                eps, out, copy)
        return x, h
    rows = table[tokens.clamp(0, table.shape[0] - 1)]
    if copy is not None:
        copy.copy_(rows)
    x = rows.float()
    return x, _next_input(x, norm, table.dtype, out)


def embed_norms(tokens: torch.Tensor, table: torch.Tensor,
                norms: Sequence[RowNorm]
                ) -> Tuple[torch.Tensor, List[torch.Tensor]]:
    """-> (x float [T, width], norm(x) in the table's type for each of one or
    two norms, which share their root mean square)"""
    if table.is_cuda:
        a, b = _two(norms)
        x, *h = require_lm_ext("embed_norms").lm_embed_norms(
            tokens, table, a, b, norms[0].n, norms[0].eps)
        return x, h
    x = table[tokens.clamp(0, table.shape[0] - 1)].float()
    return x, [norm(x).to(table.dtype) for norm in norms]


def _two(norms: Sequence[RowNorm]):
    """weights of up to two norms of the same row"""
    assert len(norms) <= 2 and all(
        v.offset == 0.0 and v.n == norms[0].n and v.eps == norms[0].eps
        for v in norms)
    w = [v.weight for v in norms]
    return (w + [None, None])[:2]


def add_branches(x: torch.Tensor, plain: Optional[torch.Tensor],
                 branches: Sequence[Tuple[torch.Tensor, torch.Tensor]],
                 scale: float, norms: Sequence[RowNorm], n: int, eps: float,
                 dtype: torch.dtype) -> List[torch.Tensor]:
    """What parallel sublayers made, in place into the float stream:
    x += plain + scale * (sum of o / rms(o) * weight over the up to two
    ``branches``). -> norm(x) in ``dtype`` for each of up to two norms.
    ``n``: true row size."""
    if x.is_cuda:
        (o1, w1), (o2, w2) = (list(branches) + [(None, None)] * 2)[:2]
        a, b = _two(norms)
        return require_lm_ext("add_branches").lm_add_branches(
            x, plain, o1, w1, o2, w2, scale, a, b, n, eps)
    if plain is not None:
        x += plain.float()
    for o, w in branches:
        v = o.float()
        x += scale * (v * _rms_inv(v, n, eps) * w.float())
    return [norm(x).to(dtype) for norm in norms]


def post_norm_add(o: torch.Tensor, bias: Optional[torch.Tensor],
                  weight: torch.Tensor, x: torch.Tensor, n: int,
                  eps: float, offset: float = 1.0,
                  norm: Optional[RowNorm] = None,
                  out: Optional[torch.Tensor] = None,
                  mix: Optional[Tuple[torch.Tensor, torch.Tensor]] = None
                  ) -> torch.Tensor:
    """x += v / rms(v) * (offset + weight), v = o + bias, in place on the
    float stream; returns x, or norm(x) of the same row size, in o's type
    (in ``out`` if given). ``n``: true row size. ``mix`` (pos, share), both
    [T, top]: a token's o is the sum of share * o[pos] over its slots."""
    if o.is_cuda:
        pos, share = mix if mix is not None else (None, None)
        if norm is not None:
            assert norm.offset == offset and norm.n == n and norm.eps == eps
        return require_lm_ext("post_norm_add").lm_post_norm_add(
            o, bias, weight, x, n, eps, offset,
            None if norm is None else norm.weight, out, pos, share)
    v = o.float()
    if mix is not None:
        v = (v[mix[0].long()] * mix[1][..., None]).sum(1)
    if bias is not None:
        v = v + bias.float()
    x += v * _rms_inv(v, n, eps) * (offset + weight.float())
    return _next_input(x, norm, o.dtype, out)


def add_norm(x: torch.Tensor, add: torch.Tensor,
             norm: Optional[RowNorm]) -> torch.Tensor:
    """x += add (one vector for all rows), in place on the float stream;
    returns norm(x) (or x) in add's type"""
    if x.is_cuda:
        w, n, eps, off = (None, x.shape[1], 0.0, 0.0) if norm is None \
            else (norm.weight, norm.n, norm.eps, norm.offset)
        return require_lm_ext("add_norm").lm_add_norm(x, add, w, off, n, eps)
    x += add.float()
    return _next_input(x, norm, add.dtype, None)


def output_norm(x: torch.Tensor, rows: Optional[torch.Tensor],
                weight: torch.Tensor, n: int, eps: float,
                scale: float = 1.0, offset: float = 1.0) -> torch.Tensor:
    """x[rows] / rms * (offset + weight) * scale in the weight's type."""
    if x.is_cuda:
        return require_lm_ext("output_norm").lm_output_norm(
            x, rows, weight, n, eps, scale, offset)
    v = x if rows is None else x[rows.long()]
    return (v * _rms_inv(v, n, eps) * (offset + weight.float()) * scale
            ).to(weight.dtype)


def linear_f32(x: torch.Tensor, w: torch.Tensor) -> torch.Tensor:
    """x @ w.T with a float result, for products that become the stream"""
    if x.is_cuda and x.dtype != torch.float32:
        return torch.mm(x, w.t(), out_dtype=torch.float32)
    return torch.nn.functional.linear(x.float(), w.float())


# codes of csrc/lm/lm_common.h
ACTIVATIONS = {"gelu_tanh": 0, "silu": 1, "relu2": 2, "none": 3, "swiglu": 4}


def activate(z: torch.Tensor, act: str) -> torch.Tensor:
    if act == "gelu_tanh":
        return torch.nn.functional.gelu(z, approximate="tanh")
    if act == "silu":
        return torch.nn.functional.silu(z)
    if act == "relu2":
        return torch.relu(z).square()
    if act == "swiglu":  # columns in pairs (gate, up)
        return torch.nn.functional.silu(z[..., ::2]) * z[..., 1::2]
    return z


def gated_mul(gate_up: torch.Tensor, bias: Optional[torch.Tensor],
              act: str) -> torch.Tensor:
    """act(gate + bg) * (up + bu); gate_up = [gate | up] columns; act:
    gelu_tanh or silu."""
    if gate_up.is_cuda:
        return require_lm_ext("gated_mul").lm_gated_mul(gate_up, bias,
                                                        ACTIVATIONS[act])
    v = gate_up.float()
    if bias is not None:
        v = v + bias.float()
    g, u = v.chunk(2, dim=-1)
    return (activate(g, act) * u).to(gate_up.dtype)


def xielu(z: torch.Tensor, coef: torch.Tensor, out: torch.Tensor) -> None:
    """coef (a, b), float: a z^2 + z / 2 for z > 0, else b (e^z - 1 - z) +
    z / 2. out [T, ff] can be a range of columns."""
    if z.is_cuda:
        require_lm_ext("xielu").lm_xielu(z, coef, out)
        return
    v = z.float()
    a, b = coef.tolist()
    out.copy_(torch.where(v > 0, a * v * v, b * (torch.expm1(v) - v))
              + 0.5 * v)


def gather_rows(src: torch.Tensor, idx: torch.Tensor) -> torch.Tensor:
    """rows of ``src`` (last dim kept, the others flattened)"""
    if src.is_cuda:
        return require_lm_ext("gather_rows").lm_gather_rows(src, idx)
    return src.reshape(-1, src.shape[-1])[idx.long()]


# --------------------------------------------------------------------- #
# latent attention
# --------------------------------------------------------------------- #
class Rotary:
    """Rotary positions: pair i turns by position * inv_freq[i], the result
    times ``gain``. Pairs are neighbours (2i, 2i+1) or, with ``half``,
    (i, i + pairs)."""

    __slots__ = ("inv_freq", "gain", "half")

    def __init__(self, inv_freq: torch.Tensor, gain: float = 1.0,
                 half: bool = False):
        self.inv_freq, self.gain, self.half = inv_freq, gain, half

    def rotate_(self, v: torch.Tensor, positions: torch.Tensor) -> None:
        """v [T, ..., >= 2 * pairs] in place (CPU equations)"""
        n = self.inv_freq.numel()
        ang = positions.float()[:, None] * self.inv_freq[None, :]
        while ang.dim() < v.dim():
            ang = ang.unsqueeze(1)
        c, s = self.gain * ang.cos(), self.gain * ang.sin()
        first, second = (slice(0, n), slice(n, 2 * n)) if self.half else \
            (slice(0, 2 * n, 2), slice(1, 2 * n, 2))
        a, b = v[..., first].float(), v[..., second].float()
        a, b = a * c - b * s, b * c + a * s
        v[..., first] = a.to(v.dtype)
        v[..., second] = b.to(v.dtype)


def yarn_frequencies(base: float, dims: int, factor: float, original: float,
                     fast: float, slow: float) -> Tuple[torch.Tensor, float]:
    """YaRN: pairs that turn fewer than ``slow`` times in ``original``
    positions are slowed by ``factor``, those that turn more than ``fast``
    times keep their frequency, a linear ramp over the dimensions in
    between. -> (float64 frequencies, gain of the rotated vectors)"""
    freq = float(base) ** (
        -2.0 * torch.arange(dims // 2, dtype=torch.float64) / dims)

    def dim_of(turns):
        return dims * math.log(original / (2.0 * math.pi * turns)) / (
            2.0 * math.log(base))

    lo = max(math.floor(dim_of(fast)), 0)
    hi = min(math.ceil(dim_of(slow)), dims - 1)
    ramp = ((torch.arange(dims // 2, dtype=torch.float64) - lo)
            / max(hi - lo, 0.001)).clamp(0.0, 1.0)
    return (freq / factor * ramp + freq * (1.0 - ramp),
            0.1 * math.log(factor) + 1.0)


def _store_latent(lat, positions, slot_mapping, rot, cp, kv_rank, eps,
                  kv_norm, cache):
    lat = lat.clone()
    c = lat[:, :cp].float()
    lat[:, :cp] = (c * _rms_inv(c, kv_rank, eps) * kv_norm.float()
                   ).to(lat.dtype)
    rot.rotate_(lat[:, cp:], positions)
    keep = slot_mapping >= 0
    cache.view(-1, lat.shape[1])[slot_mapping[keep].long()] = lat[keep]


def latent_prep(qkv: torch.Tensor, positions: torch.Tensor,
                slot_mapping: torch.Tensor, rot: Rotary,
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
    nq = heads * (dp + rp)
    lat = None if kv_norm is None else qkv[:, nq:nq + cp + rp]
    if qkv.is_cuda:
        require_lm_ext("latent_prep").lm_latent_prep(
            qkv[:, :nq], lat, None, positions, slot_mapping, rot.inv_freq,
            rot.gain, rot.half, heads, dp, rp, cp, kv_rank, eps, kv_norm,
            cache, q_abs, n_abs, None, 0)
        return
    q = qkv[:, :nq].view(-1, heads, dp + rp)
    rot.rotate_(q[..., dp:], positions)
    if n_abs:
        q_abs[..., cp:] = q[:n_abs, :, dp:]
    if lat is not None:
        _store_latent(lat, positions, slot_mapping, rot, cp, kv_rank, eps,
                      kv_norm, cache)


def latent_prep_two(cq: torch.Tensor, lat: torch.Tensor,
                    positions: torch.Tensor, slot_mapping: torch.Tensor,
                    rot: Rotary, rp: int, cp: int, kv_rank: int,
                    q_rank: int, eps: float, q_norm: torch.Tensor,
                    kv_norm: torch.Tensor, cache: torch.Tensor
                    ) -> torch.Tensor:
    """For queries that come from a latent of their own: both latents are
    normalised, the shared key part is rotated and the cache row of each
    token written. cq [T, pad of q_rank] and lat [T, cp + rp] are column
    ranges of one matrix. -> normed query latents"""
    if cq.is_cuda:
        return require_lm_ext("latent_prep").lm_latent_prep(
            None, lat, cq, positions, slot_mapping, rot.inv_freq, rot.gain,
            rot.half, 0, 0, rp, cp, kv_rank, eps, kv_norm, cache, None, 0,
            q_norm, q_rank)
    _store_latent(lat, positions, slot_mapping, rot, cp, kv_rank, eps,
                  kv_norm, cache)
    v = cq.float()
    return (v * _rms_inv(v, q_rank, eps) * q_norm.float()).to(cq.dtype)


def rotate_query(q: torch.Tensor, positions: torch.Tensor, rot: Rotary,
                 heads: int, dp: int, rp: int) -> None:
    """q [T, heads x (dp | rp)], in place"""
    if q.is_cuda:
        require_lm_ext("latent_prep").lm_latent_prep(
            q, None, None, positions, positions, rot.inv_freq, rot.gain,
            rot.half, heads, dp, rp, 32, 1, 0.0, None, None, None, 0, None,
            0)
        return
    rot.rotate_(q.view(-1, heads, dp + rp)[..., dp:], positions)


def head_gemm(a: torch.Tensor, w: torch.Tensor, out: torch.Tensor,
              gate: Optional[torch.Tensor] = None) -> None:
    """out[t, h] = w[h] @ a[t, h], times sigmoid(gate[t, h * N:]) if given;
    w [H, N, K], strided a, out and gate rows."""
    if a.is_cuda:
        require_lm_ext("head_gemm").lm_head_gemm(a, w, out, gate, None, None,
                                                 1.0, False, 0)
        return
    o = torch.matmul(a.transpose(0, 1).float(),
                     w.float().transpose(1, 2)).transpose(0, 1)
    if gate is not None:
        o = o * torch.sigmoid(gate.float()).view(o.shape)
    out.copy_(o)


def absorb_query(q: torch.Tensor, w: torch.Tensor, q_abs: torch.Tensor,
                 positions: torch.Tensor, rot: Rotary) -> None:
    """q_abs[t, h] = [w[h] @ unrotated part | rotated part] of q[t, h];
    w [H, N, K], q [T, H, K + rp], q_abs [T, H, N + rp]"""
    k, n = w.shape[2], w.shape[1]
    if q.is_cuda:
        require_lm_ext("head_gemm").lm_head_gemm(
            q, w, q_abs, None, positions, rot.inv_freq, rot.gain, rot.half,
            q.shape[2] - k)
        return
    head_gemm(q[..., :k], w, q_abs[..., :n])
    r = q[..., k:].clone()
    rot.rotate_(r, positions[:q.shape[0]])
    q_abs[..., n:] = r


def _sink_softmax(s: torch.Tensor, sink: Optional[torch.Tensor]
                  ) -> torch.Tensor:
    """softmax over the last dim, with a sink exp(sink) added to the
    denominator"""
    if sink is None:
        return torch.softmax(s, dim=-1)
    full = torch.cat([s, sink.expand(*s.shape[:-1], 1)], dim=-1)
    return torch.softmax(full, dim=-1)[..., :-1]


def latent_attention(q_abs: torch.Tensor, cache: torch.Tensor,
                     block_table: torch.Tensor, tok_seq: torch.Tensor,
                     positions: torch.Tensor, sink: Optional[torch.Tensor],
                     scale: float, window: int, cp: int,
                     max_keys: int) -> torch.Tensor:
    """Absorbed form. q_abs [n, H, cp + rp]; each token attends to the cached
    rows of its own sequence up to its position, the last ``window`` of them
    (0: all). ``sink`` [H] or None. ``max_keys``: bound on positions + 1, sizes the launch.
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
        w = _sink_softmax(s, None if sink is None else sink.float()[:, None])
        out[t] = (w @ k[:, :cp]).to(out.dtype)
    return out


PROMPT_TILE = 128     # queries per workgroup of latent_prompt
PROMPT_MAX_HEAD = 256  # largest padded key and value size it takes


def latent_prompt(q: torch.Tensor, kv: torch.Tensor, lat: torch.Tensor,
                  sink: Optional[torch.Tensor], qtiles: torch.Tensor,
                  out: torch.Tensor, heads: int, dp: int, rp: int, cp: int,
                  vp: int, window: int, scale: float,
                  gate: Optional[torch.Tensor] = None) -> None:
    """Expanded form, for prompt portions. q [T, heads * (dp + rp)]; kv
    [rows, heads * dp | heads * vp] keys and values of the gathered cache
    rows lat [rows, cp + rp]; qtiles [n, 6]: first token, tokens, first
    position, first gathered row, its position, gathered rows of the
    sequence. Writes out [T, heads, vp] at the tiles' tokens, times
    sigmoid(gate [T, heads * vp]) if given."""
    if q.is_cuda:
        require_lm_ext("latent_prompt").lm_latent_prompt(
            q, kv, lat, sink, qtiles, out, heads, dp, rp, cp, vp, window,
            scale, gate)
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
                          None if sink is None else
                          sink.float()[:, None, None])
        o = torch.einsum("hnk,khd->nhd", w, v)
        if gate is not None:
            o = o * torch.sigmoid(gate[t0:t0 + n].float()).view(o.shape)
        out[t0:t0 + n] = o.to(out.dtype)


# --------------------------------------------------------------------- #
# mixture of experts
# --------------------------------------------------------------------- #
class ExpertPlan:
    """Where a batch's T * slots slots go: share, pos [T, slots] weight and
    row of each slot (row -1: an identity expert); tok [T * slots] token of
    each row (rows in expert order); plan: tiles of up to ``rows`` rows of one
    expert."""

    __slots__ = ("share", "pos", "tok", "plan", "rows")

    def __init__(self, share, pos, tok, plan, rows):
        self.share, self.pos, self.tok = share, pos, tok
        self.plan, self.rows = plan, rows


class Routing(NamedTuple):
    """``over_all``: scores are the softmax over all router outputs, the
    choice is by score + correction (where there is one) among the ``keep``
    best of ``groups`` equal groups, and the weights are the scores;
    otherwise the largest logits, weighed by the softmax over them. The last
    ``identity`` outputs are identity experts. ``shared`` slots behind the
    chosen ones go to experts that every token takes, weighed by the sigmoid
    of one more router row."""

    top: int
    over_all: bool = False
    groups: int = 1
    keep: int = 1
    identity: int = 0
    shared: int = 0


def expert_tile_rows(n_tok: int, experts: int, top: int, dtype,
                     inner: Tuple[int, ...]) -> int:
    """rows per tile for a batch size; ``inner``: the products' inner sizes"""
    each = n_tok * top / experts
    if dtype != torch.bfloat16 or any(k % 64 for k in inner):
        return 16 if each <= 12 else 64
    if n_tok * top <= 8:  # few tiles: small column ranges fill the chip
        return 16
    if each <= 20:
        return 32
    if each <= 72:
        return 64
    return 128 if each <= 512 else 256


def _choices(z: torch.Tensor, how: Routing,
             correction: Optional[torch.Tensor]):
    """-> chosen router outputs [T, top], their weights"""
    if not how.over_all:
        z, ids = torch.topk(z, how.top, dim=-1)
        return ids, torch.softmax(z, -1)
    s = torch.softmax(z, -1)
    c = s if correction is None else s + correction
    if how.keep < how.groups:
        g = c.view(c.shape[0], how.groups, -1)
        best = g.max(-1).values.topk(how.keep, dim=-1).indices
        keep = torch.zeros(g.shape[:2], dtype=torch.bool)
        keep.scatter_(1, best, True)
        c = g.masked_fill(~keep[..., None], float("-inf")).view_as(c)
    ids = torch.topk(c, how.top, dim=-1).indices
    return ids, s.gather(1, ids)


def moe_route(h: torch.Tensor, router: torch.Tensor,
              how: Union[Routing, int], rows: int,
              correction: Optional[torch.Tensor] = None) -> ExpertPlan:
    """Experts of every token and their weights, all of it in float;
    router [outputs (+ 1 with shared slots), K]. ``how`` can be the number
    of experts alone."""
    if isinstance(how, int):
        how = Routing(how)
    if h.is_cuda:
        return ExpertPlan(*require_lm_ext("moe_route").lm_moe_route(
            h, router, how.top, rows, how.over_all, correction, how.groups,
            how.keep, how.identity, how.shared), rows)
    z = h.float() @ router.float().T
    n = router.shape[0] - (1 if how.shared else 0)
    ids, share = _choices(z[:, :n], how, correction)
    real = n - how.identity
    if how.shared:
        ids = torch.cat([ids, (real + torch.arange(how.shared)).expand(
            len(ids), -1) + how.identity], 1)
        share = torch.cat([share, torch.sigmoid(z[:, n:]).expand(
            -1, how.shared)], 1)
    # number in the plan: experts, shared ones, identities last
    flat = ids.reshape(-1)
    own = (flat >= real) & (flat < n)
    flat = torch.where(flat >= n, flat - how.identity, flat)
    flat = torch.where(own, real + how.shared, flat)
    order = torch.argsort(flat, stable=True)
    pos = torch.empty_like(order)
    pos[order] = torch.arange(order.numel())
    pos[own] = -1
    return ExpertPlan(share, pos.view(ids.shape).int(),
                      (order // ids.shape[1]).int(), flat[order], rows)


def moe_gemm(a: torch.Tensor, w: torch.Tensor, p: ExpertPlan, act: str,
             gather: bool) -> torch.Tensor:
    """out[r] = act(w[expert of row r] @ a[r]), a of row r's token with
    ``gather``; w [experts, N, K]. ``swiglu``: rows of w in pairs (gate, up),
    half as many columns."""
    n = p.tok.numel()
    if a.is_cuda:
        return require_lm_ext("moe_gemm").lm_moe_gemm(
            a, p.tok if gather else None, w, p.plan, n, p.rows,
            ACTIVATIONS[act])
    src = a[p.tok.long()] if gather else a
    out = a.new_zeros(n, w.shape[1] // (2 if act == "swiglu" else 1))
    for e in p.plan.unique().tolist():
        if e < w.shape[0]:
            at = p.plan == e
            out[at] = activate(src[at].float() @ w[e].float().T,
                               act).to(a.dtype)
    return out


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
