"""Plain, slow Nelovik: the whole design in a few dense equations.

One function per mechanism, one sequence at a time, no cache, no batching,
float64 throughout. Nothing here is shared with the serving path.

Notation: x[t] the residual, h a mixer's input, all weights [out, in].
"""

import math

import torch


def sigmoid(z):
    return 1.0 / (1.0 + torch.exp(-z))


def silu(z):
    return z * sigmoid(z)


def softplus(z):
    return torch.clamp(z, min=0.0) + torch.log1p(torch.exp(-z.abs()))


def over_rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def soft_cap(z, cap):
    return cap * torch.tanh(z / cap)


def unit(x):
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


# ---- attention ------------------------------------------------------- #
def rotate_halves(x, pos, rot):
    """x[t, ..., d]: of the first rot.dims, i turns with i + dims / 2"""
    n = rot["dims"]
    half = n // 2
    freq = torch.tensor([rot["base"] ** (-2.0 * i / n) for i in range(half)],
                        dtype=torch.float64)
    ang = pos.double()[:, None] * freq
    while ang.dim() < x.dim():
        ang = ang.unsqueeze(1)
    u, v = x[..., :half], x[..., half:n]
    return torch.cat([u * torch.cos(ang) - v * torch.sin(ang),
                      v * torch.cos(ang) + u * torch.sin(ang), x[..., n:]],
                     -1)


def block_means(x, pool):
    """x[t, ...] -> means over whole blocks of ``pool`` tokens"""
    n = x.shape[0] // pool
    return x[:n * pool].view(n, pool, *x.shape[1:]).mean(1)


def visible(n, mask):
    """[query, token] and [query, block]"""
    i = torch.arange(n)[:, None]
    j = torch.arange(n)[None, :]
    tokens = (j <= i) & (i - j < mask["size"])
    last = torch.arange(n // mask["pool"])[None, :] * mask["pool"] \
        + mask["pool"] - 1
    return tokens, last <= i - mask["size"]


def weigh(scores, see, sink):
    """softmax over the visible keys, exp(sink) more in the denominator"""
    s = scores.masked_fill(~see, -math.inf)
    top = torch.clamp(s.max(-1, keepdim=True).values, min=float(sink))
    e = torch.exp(s - top)
    return e / (e.sum(-1, keepdim=True) + torch.exp(sink - top))


def attend(q, k, v, m, sinks):
    """q [t, H, d], k [t, G, d], v [t, G, dv] -> [t, H * dv]"""
    n, heads = q.shape[:2]
    per = heads // k.shape[1]
    pool = m["mask"]["pool"]
    keys = torch.cat([block_means(k, pool), k])
    vals = torch.cat([block_means(v, pool), v])
    tokens, blocks = visible(n, m["mask"])
    see = torch.cat([blocks, tokens], 1)
    out = []
    for a in range(heads):
        s = soft_cap((q[:, a] @ keys[:, a // per].T) * m["scale"],
                     m["softcap"])
        out.append(weigh(s, see, sinks[a]) @ vals[:, a // per])
    return torch.cat(out, -1)


def window_attention(h, w, m, eps):
    n = h.shape[0]
    pos = torch.arange(n)
    q = over_rms(h @ w["q"].T + w["q.b"], eps) * w["q.norm"]
    k = over_rms(h @ w["k"].T + w["k.b"], eps) * w["k.norm"]
    v = h @ w["v"].T + w["v.b"]
    q = rotate_halves(q.view(n, m["heads"], m["dim"]), pos, m["rot"])
    k = rotate_halves(k.view(n, m["kv_heads"], m["dim"]), pos, m["rot"])
    o = attend(q, k, v.view(n, m["kv_heads"], m["vdim"]), m, w["sink"])
    return o @ w["o"].T


# ---- recurrences ----------------------------------------------------- #
def causal_conv(x, taps, bias=None):
    """x [t, c], taps [c, n]: taps[:, n - 1 - d] goes with x[t - d]"""
    n = taps.shape[1]
    out = torch.zeros_like(x)
    for d in range(min(n, x.shape[0])):  # d tokens back
        out[d:] += x[:x.shape[0] - d] * taps[:, n - 1 - d]
    return out if bias is None else out + bias


def delta_scan(q, k, v, decay, beta, state=None):
    """one head: q, k [t, d], v [t, dv], decay, beta [t] -> (o [t, dv], last
    state [d, dv])"""
    s = torch.zeros(q.shape[1], v.shape[1], dtype=q.dtype) \
        if state is None else state.clone()
    out = torch.zeros_like(v)
    for t in range(q.shape[0]):
        s = decay[t] * s
        s = s + torch.outer(k[t], beta[t] * (v[t] - s.T @ k[t]))
        out[t] = s.T @ q[t]
    return out, s


def delta_rule(h, w, m, eps):
    n, heads = h.shape[0], m["heads"]
    per = heads // m["kv_heads"]
    q, k, v = (silu(causal_conv(h @ w[x].T, w[x + ".conv"])) for x in "qkv")
    q = unit(q.view(n, m["kv_heads"], m["dim"])) * m["dim"] ** -0.5
    k = unit(k.view(n, m["kv_heads"], m["dim"]))
    v = v.view(n, heads, m["vdim"])
    beta = sigmoid(h @ w["b"].T)
    decay = torch.exp(-torch.exp(w["A_log"])
                      * softplus(h @ w["a"].T + w["dt_bias"]))
    o = torch.stack([delta_scan(q[:, a // per], k[:, a // per], v[:, a],
                                decay[:, a], beta[:, a])[0]
                     for a in range(heads)], 1)
    o = (over_rms(o, eps) * w["norm"]).reshape(n, -1)
    return (o * silu(h @ w["g"].T)) @ w["o"].T


def state_scan(x, b, c, dt, rate, d, state=None):
    """one head: x [t, p], b, c [t, N], dt [t], rate and d numbers ->
    (y [t, p], last state [N, p])"""
    s = torch.zeros(b.shape[1], x.shape[1], dtype=x.dtype) \
        if state is None else state.clone()
    out = torch.zeros_like(x)
    for t in range(x.shape[0]):
        s = torch.exp(-rate * dt[t]) * s + dt[t] * torch.outer(b[t], x[t])
        out[t] = s.T @ c[t] + d * x[t]
    return out, s


def state_space(h, w, m, eps):
    n, heads, p = h.shape[0], m["heads"], m["vdim"]
    inner, gn = heads * p, m["groups"] * m["state"]
    per = heads // m["groups"]
    z, xbc, dt = torch.split(h @ w["in"].T, [inner, inner + 2 * gn, heads],
                             -1)
    xbc = silu(causal_conv(xbc, w["conv"], w["conv.b"]))
    x, b, c = torch.split(xbc, [inner, gn, gn], -1)
    x = x.view(n, heads, p)
    b, c = (y.view(n, m["groups"], m["state"]) for y in (b, c))
    dt = softplus(dt + w["dt_bias"])
    y = torch.cat([state_scan(x[:, a], b[:, a // per], c[:, a // per],
                              dt[:, a], torch.exp(w["A_log"][a]),
                              w["D"][a])[0] for a in range(heads)], -1)
    return gated_norm(y, z, w["norm"], m["norm_groups"], eps) @ w["o"].T


def gated_norm(y, z, weight, parts, eps):
    y = (y * silu(z)).view(y.shape[0], parts, -1)
    return over_rms(y, eps).reshape(z.shape) * weight


def parallel(h, w, m, eps):
    left = window_attention(h, sub(w, "left."), m["left"], eps)
    right = state_space(h, sub(w, "right."), m["right"], eps)
    return 0.5 * (over_rms(left, eps) * w["left.out"]
                  + over_rms(right, eps) * w["right.out"])


# ---- feed-forward ---------------------------------------------------- #
def xielu(z, p, q):
    up = softplus(p) * z * z
    down = (0.5 + softplus(q)) * (torch.expm1(z) - z)
    return torch.where(z > 0, up, down) + 0.5 * z


def dense(h, w):
    return xielu(h @ w["up"].T, w["act"][0], w["act"][1]) @ w["down"].T


# ---- the model ------------------------------------------------------- #
MIXERS = {"parallel": parallel, "delta": delta_rule, "delta_2": delta_rule}


def sub(state, prefix):
    return {k[len(prefix):]: v for k, v in state.items()
            if k.startswith(prefix)}


def forward(cfg, state, tokens, collect=None):
    """-> logits [n, vocab]; ``collect`` receives the residual after every
    layer."""
    state = {k: v.double() for k, v in state.items()}
    eps = cfg["norm"]["eps"]
    x = state["embed"][torch.as_tensor(tokens)]
    for i, spec in enumerate(cfg["layers"]):
        w = sub(state, "l{}.".format(i))
        y = MIXERS[spec["type"]](over_rms(x, eps) * w["norm1"],
                                 sub(w, "mix."), spec["mixer"], eps)
        if spec.get("mlp") is not None:
            y = y + dense(over_rms(x, eps) * w["norm2"], sub(w, "mlp."))
        x = x + y
        if collect is not None:
            collect.append(x)
    return (over_rms(x, eps) * state["final.norm"]) @ state["head"].T
