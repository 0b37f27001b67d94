"""Plain, slow Kakipel: the whole design in a few dense equations.

One function per mechanism, one sequence at a time, no cache, no batching,
float64 throughout. Nothing here is shared with the serving path.

Notation: x[t] residual stream, h a sublayer's input, all weights [out, in].
"""

import math

import torch


def rms_norm(x, w, eps):
    return w * x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def sigmoid(z):
    return 1.0 / (1.0 + torch.exp(-z))


def silu(z):
    return z * sigmoid(z)


def relu_squared(z):
    return torch.where(z > 0, z * z, torch.zeros_like(z))


def frequencies(rot):
    """-> (angle per position of each pair, factor of cos and sin)"""
    d, base, s = rot["dims"], rot["base"], rot.get("scaling")
    freq = [base ** (-2.0 * i / d) for i in range(d // 2)]
    if s is None:
        return torch.tensor(freq, dtype=torch.float64), 1.0

    def dim_of(turns):  # the dimension that turns so often in `original`
        return (d * math.log(s["original"] / (2.0 * math.pi * turns))
                / (2.0 * math.log(base)))

    lo = max(math.floor(dim_of(s["fast"])), 0)
    hi = min(math.ceil(dim_of(s["slow"])), d - 1)
    out = []
    for i, f in enumerate(freq):
        r = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(f / s["factor"] * r + f * (1.0 - r))
    return (torch.tensor(out, dtype=torch.float64),
            0.1 * math.log(s["factor"]) + 1.0)


def rotate_half(x, pos, rot):
    """x[t, ..., d]: of the first rot.dims, i turns with i + dims/2"""
    freq, gain = frequencies(rot)
    n = freq.numel()
    ang = pos.double()[:, None] * freq
    while ang.dim() < x.dim():
        ang = ang.unsqueeze(1)
    c, s = gain * torch.cos(ang), gain * torch.sin(ang)
    u, v = x[..., :n], x[..., n:2 * n]
    return torch.cat([u * c - v * s, v * c + u * s, x[..., 2 * n:]], -1)


def softmax_rows(s):
    e = torch.exp(s - s.max(-1, keepdim=True).values)
    return e / e.sum(-1, keepdim=True)


def latent_attention(h, w, m, eps):
    n = h.shape[0]
    heads, dim, rd, vd = m["heads"], m["dim"], m["rot_dim"], m["vdim"]
    pos = torch.arange(n)
    cq = rms_norm(h @ w["dq"].T, w["dq.norm"], eps)
    q = (cq @ w["uq"].T).view(n, heads, dim + rd)
    z = h @ w["dkv"].T
    c = rms_norm(z[:, :m["kv_rank"]], w["dkv.norm"], eps)
    kr = rotate_half(z[:, m["kv_rank"]:], pos, m["rot"])
    k = (c @ w["uk"].T).view(n, heads, dim)
    v = (c @ w["uv"].T).view(n, heads, vd)
    qr = rotate_half(q[..., dim:], pos, m["rot"])
    later = pos[None, :] > pos[:, None]
    out = torch.zeros(n, heads, vd, dtype=h.dtype)
    for a in range(heads):
        s = (q[:, a, :dim] @ k[:, a].T + qr[:, a] @ kr.T) * m["scale"]
        out[:, a] = softmax_rows(s.masked_fill(later, -math.inf)) @ v[:, a]
    out = out.reshape(n, heads * vd) * sigmoid(h @ w["g"].T)
    return out @ w["o"].T


def dense_ff(h, w):
    return (silu(h @ w["gate"].T) * (h @ w["up"].T)) @ w["down"].T


def route(h, w_router, top):
    """-> chosen experts [n, top] and their weights"""
    z = h @ w_router.T
    chosen = torch.sort(z, dim=-1, descending=True, stable=True)
    return chosen.indices[:, :top], softmax_rows(chosen.values[:, :top])


def expert_ff(h, up, down):
    return relu_squared(h @ up.T) @ down.T


def mixture_ff(h, w, mlp):
    ids, p = route(h, w["router"], mlp["router"]["top"])
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, pe in zip(ids[t].tolist(), p[t]):
            out[t] += pe * expert_ff(h[t], w["e{}.up".format(e)],
                                     w["e{}.down".format(e)])
    return out


def sub(state, prefix):
    return {k[len(prefix):]: v for k, v in state.items()
            if k.startswith(prefix)}


def layer(x, state, n, spec, eps):
    p = "l{}.".format(n)
    h = rms_norm(x, state[p + "norm1"], eps)
    o = latent_attention(h, sub(state, p + "mix."), spec["mixer"], eps)
    x = x + rms_norm(o, state[p + "norm1b"], eps)
    mlp = spec.get("mlp")
    if mlp is not None:
        h = rms_norm(x, state[p + "norm2"], eps)
        w = sub(state, p + "mlp.")
        o = dense_ff(h, w) if mlp["kind"] == "dense" else \
            mixture_ff(h, w, mlp)
        x = x + rms_norm(o, state[p + "norm2b"], eps)
    return x


def loop_entry(x, x0, w_in, step):
    return torch.cat([x, x0], -1) @ w_in.T + step


def schedule(cfg):
    """layer runs in order: (layer, pass entered right before it or None)"""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if loop is None:
        return [(i, None) for i in range(n)]
    out = [(i, None) for i in range(loop["start"])]
    for t in range(loop["times"]):
        out += [(i, t if i == loop["start"] else None)
                for i in range(loop["start"], loop["stop"])]
    return out + [(i, None) for i in range(loop["stop"], n)]


def forward(cfg, state, tokens, collect=None):
    """-> logits [n, vocab]; ``collect`` receives x after every layer run."""
    state = {k: v.double() for k, v in state.items()}
    eps = cfg["norm"]["eps"]
    x = x0 = state["embed"][torch.as_tensor(tokens)]
    for i, t in schedule(cfg):
        if t is not None:
            x = loop_entry(x, x0, state["loop.in"], state["loop.step"][t])
        x = layer(x, state, i, cfg["layers"][i], eps)
        if collect is not None:
            collect.append(x.clone())
    return rms_norm(x, state["final.norm"], eps) @ state["head"].T
