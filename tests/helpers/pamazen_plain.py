"""Plain, slow Pamazen: the whole design in a few dense equations.

One function per mechanism, one sequence at a time, no cache, no batching,
float64 throughout. Nothing here is shared with the serving path.

Notation: X[s][t] stream s of the residual, h a sublayer's input, all weights
[out, in].
"""

import math

import torch


def sigmoid(z):
    return 1.0 / (1.0 + torch.exp(-z))


def silu(z):
    return z * sigmoid(z)


def over_rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def soft_cap(z, cap):
    return cap * torch.tanh(z / cap)


# ---- attention ------------------------------------------------------- #
def frequencies(rot):
    factor = rot.get("scaling", {}).get("factor", 1.0)
    d = rot["dims"]
    return torch.tensor([rot["base"] ** (-2.0 * i / d) / factor
                         for i in range(d // 2)], dtype=torch.float64)


def rotate_neighbours(x, pos, rot):
    """x[t, ..., d]: of the first rot.dims, 2i turns with 2i + 1"""
    freq = frequencies(rot)
    n = rot["dims"]
    ang = pos.double()[:, None] * freq
    while ang.dim() < x.dim():
        ang = ang.unsqueeze(1)
    out = x.clone()
    u, v = x[..., 0:n:2], x[..., 1:n:2]
    out[..., 0:n:2] = u * torch.cos(ang) - v * torch.sin(ang)
    out[..., 1:n:2] = v * torch.cos(ang) + u * torch.sin(ang)
    return out


def visible(n, mask):
    """[query, key]: causal, with a mask also the last ``size`` keys and the
    first ``keep_first`` ones"""
    i = torch.arange(n)[:, None]
    j = torch.arange(n)[None, :]
    see = j <= i
    if mask is not None:
        see = see & ((i - j < mask["size"]) | (j < mask["keep_first"]))
    return see


def weigh(scores, see, sink):
    """softmax over the visible keys, exp(sink) more in the denominator"""
    s = scores.masked_fill(~see, -math.inf)
    top = torch.clamp(s.max(-1, keepdim=True).values, min=float(sink))
    e = torch.exp(s - top)
    return e / (e.sum(-1, keepdim=True) + torch.exp(sink - top))


def attend(q, k, v, m, mask, cap, sinks):
    """q [t, H, d], k [t, G, d], v [t, G, dv] -> [t, H * dv]"""
    n, heads = q.shape[:2]
    per = heads // k.shape[1]
    see = visible(n, mask)
    out = []
    for a in range(heads):
        s = (q[:, a] @ k[:, a // per].T) * m["scale"]
        if cap is not None:
            s = soft_cap(s, cap)
        out.append(weigh(s, see, sinks[a]) @ v[:, a // per])
    return torch.cat(out, -1)


def attention(h, w, m, first_values):
    """-> (output, this layer's own values). ``first_values``: those of the
    first layer that mixes, or None."""
    n = h.shape[0]
    pos = torch.arange(n)
    q = (h @ w["q"].T).view(n, m["heads"], m["dim"])
    k = (h @ w["k"].T).view(n, m["kv_heads"], m["dim"])
    own = v = (h @ w["v"].T).view(n, m["kv_heads"], m["vdim"])
    if m.get("v_mix") and first_values is not None:
        v = (1.0 - w["vmix"]) * v + w["vmix"] * first_values
    q = rotate_neighbours(q, pos, m["rot"])
    k = rotate_neighbours(k, pos, m["rot"])
    o = attend(q, k, v, m, None, None,
               torch.zeros(m["heads"], dtype=h.dtype))
    return o @ w["o"].T, own


def window_attention(h, w, m, eps):
    n = h.shape[0]
    q = (h @ w["q"].T).view(n, m["heads"], m["dim"])
    k = (h @ w["k"].T).view(n, m["kv_heads"], m["dim"])
    o = attend(over_rms(q, eps) * w["q.norm"], over_rms(k, eps) * w["k.norm"],
               k, m, m["mask"], m["softcap"], w["sink"])
    return o @ w["o"].T


# ---- delta rule ------------------------------------------------------ #
def delta_scan(r, k, v, decay, rate, state=None):
    """one head: r, k, v, decay, rate [t, d] -> (o [t, d], last state)"""
    n, d = r.shape
    s = torch.zeros(d, d, dtype=r.dtype) if state is None else state.clone()
    u = k / torch.sqrt((k * k).sum(-1, keepdim=True) + 1e-6)
    out = torch.zeros(n, d, dtype=r.dtype)
    for t in range(n):
        s = (decay[t][:, None] * s
             - torch.outer(rate[t] * u[t], u[t] @ s)
             + torch.outer(k[t], v[t]))
        out[t] = s.T @ r[t]
    return out, s


def delta_rule(h, w, m, eps):
    n, heads, d = h.shape[0], m["heads"], m["dim"]

    def per_head(x):
        return x.view(n, heads, d)

    decay = torch.exp(-math.exp(-0.5) * sigmoid(
        torch.tanh(h @ w["w1"].T) @ w["w2"].T + w["w0"]))
    rate = sigmoid(h @ w["a"].T + w["a.b"])
    r, k, v = (per_head(h @ w[x].T) for x in "rkv")
    o = torch.stack([delta_scan(r[:, a], k[:, a], v[:, a],
                                per_head(decay)[:, a],
                                per_head(rate)[:, a])[0]
                     for a in range(heads)], 1)
    o = over_rms(o, eps).reshape(n, heads * d)
    return (o * w["norm"] * sigmoid(h @ w["g"].T)) @ w["o"].T


def parallel(h, w, m, eps):
    return (m["left_scale"] * window_attention(h, sub(w, "left."), m["left"],
                                               eps)
            + m["right_scale"] * delta_rule(h, sub(w, "right."), m["right"],
                                            eps))


# ---- feed-forward ---------------------------------------------------- #
def expert(h, w, p):
    return (silu(h @ w[p + "gate"].T) * (h @ w[p + "up"].T)) \
        @ w[p + "down"].T


def route(h, w_router, correction, router):
    """-> chosen outputs [n, top] and their weights"""
    s = torch.softmax(h @ w_router.T, -1)
    c = s + correction
    groups = router.get("groups")
    if groups is not None:
        g = c.view(c.shape[0], groups["count"], -1)
        best = torch.sort(g.max(-1).values, dim=-1, descending=True,
                          stable=True).indices
        keep = torch.zeros(g.shape[:2], dtype=torch.bool)
        keep.scatter_(1, best[:, :groups["keep"]], True)
        c = g.masked_fill(~keep[..., None], -math.inf).reshape(c.shape)
    ids = torch.sort(c, dim=-1, descending=True, stable=True).indices
    ids = ids[:, :router["top"]]
    return ids, s.gather(1, ids)


def mixture(h, w, mlp):
    r = mlp["router"]
    ids, p = route(h, w["router"], w["correction"], r)
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, pe in zip(ids[t].tolist(), p[t]):
            out[t] += pe * (h[t] if e >= r["experts"] else
                            expert(h[t], w, "e{}.".format(e)))
    if mlp.get("shared") is not None:
        out = out + sigmoid(h @ w["shared.sg"].T) * expert(h, w, "shared.")
    return out


# ---- the model ------------------------------------------------------- #
def sub(state, prefix):
    return {k[len(prefix):]: v for k, v in state.items()
            if k.startswith(prefix)}


def into(streams, w):
    return sum(w["in"][s] * x for s, x in enumerate(streams))


def out_of(streams, y, w, m):
    return [sum(w["mix"][s, t] * x for s, x in enumerate(streams))
            + m * w["out"][t] * y for t in range(len(streams))]


def forward(cfg, state, tokens, collect=None):
    """-> logits [n, vocab]; ``collect`` receives the sum of the streams
    after every layer."""
    state = {k: v.double() for k, v in state.items()}
    eps, m = cfg["norm"]["eps"], cfg["residual_mult"]
    x = state["embed"][torch.as_tensor(tokens)]
    streams = [x.clone() for _ in range(cfg["streams"])]
    first = None
    for i, spec in enumerate(cfg["layers"]):
        w = sub(state, "l{}.".format(i))
        hc = sub(w, "hc1.")
        h = over_rms(into(streams, hc), eps) * w["norm1"]
        if spec["type"] == "attention":
            y, own = attention(h, sub(w, "mix."), spec["mixer"], first)
            if spec["mixer"].get("v_mix") and first is None:
                first = own
        else:
            y = parallel(h, sub(w, "mix."), spec["mixer"], eps)
        streams = out_of(streams, y, hc, m)
        if spec.get("mlp") is not None:
            hc = sub(w, "hc2.")
            h = over_rms(into(streams, hc), eps) * w["norm2"]
            streams = out_of(streams, mixture(h, sub(w, "mlp."),
                                              spec["mlp"]), hc, m)
        if collect is not None:
            collect.append(sum(streams))
    h = over_rms(sum(streams), eps) * state["final.norm"]
    return soft_cap(h @ state["head"].T, cfg["logit_softcap"])
