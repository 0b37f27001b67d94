"""Plain, slow Bimipel: the whole design in a few dense equations.

One function per mechanism, one sequence at a time, no cache, no batching,
float64 throughout. Nothing here is shared with the serving path.

Notation: x[t] residual stream, h the sublayer's input (= x), all weights
[out, in].
"""

import math

import torch


def rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def norm_zero_centred(x, w, eps):
    return rms(x, eps) * (1.0 + w)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + torch.tanh(
        math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def sigmoid(z):
    return 1.0 / (1.0 + torch.exp(-z))


def softplus(z):
    return torch.logaddexp(z, torch.zeros_like(z))


def rotate_pairs(x, pos, base):
    """x[t, ..., d]: neighbours (2i, 2i+1) turn by pos * base^(-2i/d)."""
    d = x.shape[-1]
    i = torch.arange(d // 2, dtype=x.dtype)
    ang = pos.to(x.dtype)[:, None] * base ** (-2.0 * i / d)
    while ang.dim() < x.dim():
        ang = ang.unsqueeze(1)
    u, v = x[..., 0::2], x[..., 1::2]
    out = torch.empty_like(x)
    out[..., 0::2] = u * torch.cos(ang) - v * torch.sin(ang)
    out[..., 1::2] = v * torch.cos(ang) + u * torch.sin(ang)
    return out


def window_mask(n, size):
    i = torch.arange(n)[:, None]
    j = torch.arange(n)[None, :]
    return (i - j >= 0) & (i - j < size)


def softmax_with_sink(scores, mask, sink):
    """scores [n, m], one head; the sink only adds exp(sink) below."""
    s = scores.masked_fill(~mask, float("-inf"))
    top = torch.maximum(s.max(-1, keepdim=True).values, sink)
    e = torch.exp(s - top)
    return e / (e.sum(-1, keepdim=True) + torch.exp(sink - top))


def latent_and_rotated_key(h, w, m, eps):
    """-> (c [n, kv_rank], rotated shared key part [n, rot_dim])"""
    pos = torch.arange(h.shape[0])
    z = h @ w["dkv"].T
    c = rms(z[:, :m["kv_rank"]], eps) * w["dkv.norm"]
    kr = rotate_pairs(z[:, m["kv_rank"]:], pos, m["rot"]["base"])
    return c, kr


def latent_attention(h, w, m, c, kr):
    n = h.shape[0]
    heads, dim, rd, vd = m["heads"], m["dim"], m["rot_dim"], m["vdim"]
    pos = torch.arange(n)
    q = (h @ w["q"].T).view(n, heads, dim + rd)
    k = (c @ w["uk"].T).view(n, heads, dim)
    v = (c @ w["uv"].T).view(n, heads, vd)
    qr = rotate_pairs(q[..., dim:], pos, m["rot"]["base"])
    mask = window_mask(n, m["mask"]["size"])
    out = torch.zeros(n, heads, vd, dtype=h.dtype)
    for a in range(heads):
        s = (q[:, a, :dim] @ k[:, a].T + qr[:, a] @ kr.T) * m["scale"]
        out[:, a] = softmax_with_sink(s, mask, w["sink"][a]) @ v[:, a]
    return out.reshape(n, heads * vd) @ w["o"].T


def causal_conv(z, w, b):
    """z [n, ch], w [ch, taps]; the last column meets the current token."""
    n, taps = z.shape[0], w.shape[1]
    zp = torch.cat([torch.zeros(taps - 1, z.shape[1], dtype=z.dtype), z])
    return sum(zp[j:j + n] * w[:, j] for j in range(taps)) + b


def block_linear(u, w, b):
    """u [n, blocks*k], w [blocks, k, k]"""
    k = w.shape[1]
    return torch.cat([u[:, i * k:(i + 1) * k] @ w[i].T + b[i]
                      for i in range(w.shape[0])], -1)


def gated_linear_recurrence(u, r, i, lam):
    log_a = -8.0 * r * softplus(lam)
    a = torch.exp(log_a)
    g = torch.sqrt(1.0 - a * a) * i * u
    s = torch.zeros(u.shape[1], dtype=u.dtype)
    out = torch.empty_like(u)
    for t in range(u.shape[0]):
        s = a[t] * s + g[t]
        out[t] = s
    return out


def rglru(h, w):
    y = gelu_tanh(h @ w["y"].T + w["y.b"])
    u = causal_conv(h @ w["x"].T + w["x.b"], w["conv"], w["conv.b"])
    r = sigmoid(block_linear(u, w["ra"], w["ra.b"]))
    i = sigmoid(block_linear(u, w["ri"], w["ri.b"]))
    return (gated_linear_recurrence(u, r, i, w["lam"]) * y) @ w["o"].T


def feed_forward(h, w):
    g = gelu_tanh(h @ w["gate"].T + w["gate.b"])
    return (g * (h @ w["up"].T + w["up.b"])) @ w["down"].T + w["down.b"]


def sub(state, prefix):
    return {k[len(prefix):]: v for k, v in state.items()
            if k.startswith(prefix)}


def forward(cfg, state, tokens, collect=None):
    """-> logits [n, vocab]; ``collect`` receives x after every layer."""
    state = {k: v.double() for k, v in state.items()}
    eps = cfg["norm"]["eps"]
    x = state["embed"][torch.as_tensor(tokens)]
    kept = {}
    for n, layer in enumerate(cfg["layers"]):
        p = "l{}.".format(n)
        w, m = sub(state, p + "mix."), layer["mixer"]
        if layer["type"] == "latent_attention":
            if m.get("kv_from") is None:
                kept[n] = latent_and_rotated_key(x, w, m, eps)
                c, kr = kept[n]
            else:
                c, kr = kept[m["kv_from"]]
            o = latent_attention(x, w, m, c, kr)
        elif layer["type"] == "rglru":
            o = rglru(x, w)
        else:
            raise ValueError(layer["type"])
        x = x + norm_zero_centred(o, state[p + "norm1"], eps)
        if layer["mlp"] is not None:
            o = feed_forward(x, sub(state, p + "mlp."))
            x = x + norm_zero_centred(o, state[p + "norm2"], eps)
        if collect is not None:
            collect.append(x.clone())
    x = norm_zero_centred(x, state["final.norm"], eps)
    return x @ state["embed"].T * cfg["logit_scale"]
