"""Small Pamazen configurations and weights for the tests."""

import torch


def attn(heads=4, kv=2, dim=12, rot=6, vdim=10, base=500.0, factor=3.0,
         scale=0.3, v_mix=True):
    return {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim,
            "scale": scale, "v_mix": v_mix,
            "rot": {"base": base, "dims": rot, "scaling": {"factor": factor}}}


def left(heads=6, kv=2, dim=20, size=11, keep=3, cap=6.0, scale=0.25):
    return {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": dim,
            "scale": scale, "softcap": cap,
            "mask": {"size": size, "keep_first": keep}}


def parallel(lft=None, heads=2, dim=24, rank=5, scales=(0.8, 1.3)):
    """``rank`` is no key of the configuration: the decay's tensors have it"""
    return {"left": lft or left(), "right": {"heads": heads, "dim": dim},
            "left_scale": scales[0], "right_scale": scales[1], "_rank": rank}


def moe(experts=6, top=2, ff=20, identity=2, groups=(4, 3), shared=28):
    return {"kind": "moe", "expert": {"ff": ff}, "shared": {"ff": shared},
            "router": {"experts": experts, "top": top, "identity": identity,
                       "groups": {"count": groups[0], "keep": groups[1]}}}


def layer(mixer, mlp=None):
    return {"type": "parallel" if "left" in mixer else "attention",
            "mixer": mixer, "mlp": mlp}


def config(layers, vocab=83, width=44, eps=1e-4, streams=3, mult=0.7,
           cap=9.0):
    return {"architecture": "Pamazen", "layers": layers, "vocab": vocab,
            "width": width, "norm": {"eps": eps}, "streams": streams,
            "residual_mult": mult, "logit_softcap": cap}


# name -> configuration; together they take every branch and unequal sizes,
# also sizes of one
CONFIGS = {
    "mixed": lambda: config([
        layer(attn(v_mix=False, vdim=7, heads=3, kv=3), moe()),
        layer(parallel(), moe(5, 3, 24, 1, (2, 1), 60)),
        layer(attn(heads=6, dim=8, rot=8, scale=0.45)),
        layer(attn(dim=16, rot=2, base=77.0, factor=1.0),
              moe(7, 1, 33, 2, (3, 2), 12))]),
    # one stream, one head, no group is left out, no identity expert, a
    # window of one token (a head of one channel over its root mean square is
    # near +-1: a large eps keeps it from amplifying)
    "ones": lambda: config([
        layer(parallel(left(1, 1, 40, 1, 1, 30.0), 1, 1, 1)),
        layer(attn(1, 1, 34, 2, 1), moe(3, 3, 1, 0, (1, 1), 1)),
        layer(parallel(left(17, 1, 4, 7, 0), 3, 40, 70), moe(1, 1, 5, 1,
                                                             (2, 2), 9))],
        vocab=130, width=70, eps=0.05, streams=1, mult=1.0),
    # sizes that the tiled products take; the first layer mixes
    "aligned": lambda: config([
        layer(attn(8, 2, 32, 16, 64, base=1e4), moe(10, 3, 64, 2, (3, 2),
                                                    128)),
        layer(parallel(left(4, 4, 64, 24, 5, 15.0, 0.125), 2, 64, 32),
              moe(8, 4, 128, 0, (4, 2), 64)),
        layer(attn(4, 2, 96, 64, 64, scale=0.1), moe(6, 2, 64, 6, (2, 2),
                                                     64))],
        vocab=96, width=64, eps=1e-6, streams=4, mult=0.5, cap=20.0),
    # no layer with attention over everything; as many streams as there can be
    "windows": lambda: config([
        layer(parallel(left(2, 1, 130, 40, 2)), moe(3, 2, 30, 1, (4, 3), 31)),
        layer(parallel(left(5, 5, 9, 3, 9), 1, 130, 33, (-1.0, 0.5)))],
        vocab=64, width=32, streams=8),
}


def public(cfg):
    """the configuration as a config.json has it"""
    out = {k: v for k, v in cfg.items() if k != "layers"}
    out["layers"] = [dict(lay, mixer={k: v for k, v in lay["mixer"].items()
                                      if not k.startswith("_")})
                     for lay in cfg["layers"]]
    return out


def attention_shapes(m, w, window=False):
    h, g, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    out = {"q": (h * d, w), "k": (g * d, w), "o": (w, h * dv)}
    if window:
        out.update({"q.norm": (d,), "k.norm": (d,), "sink": (h,)})
    else:
        out["v"] = (g * dv, w)
        if m["v_mix"]:
            out["vmix"] = ()
    return out


def delta_shapes(m, w, rank):
    n = m["heads"] * m["dim"]
    out = {k: (n, w) for k in "rkvga"}
    out.update({"a.b": (n,), "w0": (n,), "w1": (rank, w), "w2": (n, rank),
                "norm": (n,), "o": (w, n)})
    return out


def moe_shapes(f, w):
    r = f["router"]
    n = r["experts"] + r["identity"]
    out = {"router": (n, w), "correction": (n,), "shared.sg": (1, w)}
    for p, e in [("e{}.".format(k), f["expert"]["ff"])
                 for k in range(r["experts"])] + [
                     ("shared.", f["shared"]["ff"])]:
        out.update({p + "gate": (e, w), p + "up": (e, w), p + "down": (w, e)})
    return out


def shapes(cfg):
    """checkpoint tensor names and shapes, from the configuration alone"""
    w, s = cfg["width"], cfg["streams"]
    out = {"embed": (cfg["vocab"], w), "head": (cfg["vocab"], w),
           "final.norm": ()}
    for n, lay in enumerate(cfg["layers"]):
        m, p = lay["mixer"], "l{}.".format(n)
        if "left" in m:
            mix = {"left." + k: v for k, v in
                   attention_shapes(m["left"], w, True).items()}
            mix.update({"right." + k: v for k, v in delta_shapes(
                m["right"], w, m["_rank"]).items()})
        else:
            mix = attention_shapes(m, w)
        out.update({p + "mix." + k: v for k, v in mix.items()})
        for q in (1, 2) if lay["mlp"] else (1,):
            out[p + "norm{}".format(q)] = ()
            hc = p + "hc{}.".format(q)
            out.update({hc + "in": (s,), hc + "out": (s,),
                        hc + "mix": (s, s)})
        if lay["mlp"]:
            out.update({p + "mlp." + k: v for k, v in
                        moe_shapes(lay["mlp"], w).items()})
    return out


def random_tensor(name, s, gen, sharp=2.5):
    """queries and keys strong enough (``sharp``) that single keys stand out;
    what is added or weighs something is neither small nor alike"""
    t = torch.randn(s, generator=gen)
    leaf = name.split(".")[-1]
    if leaf in ("in", "out"):
        return 0.6 + 0.3 * t
    if leaf == "mix" and len(s) == 2:  # of a hyper-connection
        return 0.8 * torch.eye(s[0]) + 0.2 * t
    if leaf.startswith("norm"):
        return 1.0 + 0.3 * t
    if leaf == "vmix":
        return torch.tensor(0.4) + 0.1 * t
    if leaf == "correction":
        return 0.3 * t
    if name.endswith("right.w0"):
        return t - 1.0
    if leaf == "embed":
        return t
    if len(s) == 1:
        return t
    if leaf in ("q", "w1"):
        t = t * sharp
    return t * s[-1] ** -0.5


def weights(cfg, seed=0, sharp=2.5, decided=False):
    """``decided``: no routing is a close call, whatever the rounding. A few
    coordinates of the streams, one per router output, are set by the token
    alone (sublayers do not touch them but for the identity experts, which
    keep their order); the routers read only these, and the corrections come
    in steps larger than any score."""
    gen = torch.Generator().manual_seed(seed)
    out = {k: random_tensor(k, s, gen, sharp)
           for k, s in shapes(cfg).items()}
    if decided:
        _decide(cfg, out, gen)
    return {k: v.to(torch.bfloat16) for k, v in out.items()}


def _decide(cfg, st, gen):
    n = max(lay["mlp"]["router"]["experts"] + lay["mlp"]["router"]["identity"]
            for lay in cfg["layers"] if lay["mlp"])
    assert 0 < n <= cfg["width"] // 3
    levels = 1.5 * (torch.arange(n) - (n - 1) / 2)
    for v in range(cfg["vocab"]):
        st["embed"][v, :n] = levels[torch.randperm(n, generator=gen)]
    for k, v in st.items():
        leaf = k.split(".")[-1]
        if leaf in ("o", "down"):
            v[:n] = 0
        elif leaf in ("in", "out", "mix"):
            v.abs_()
        elif leaf == "correction":
            v.copy_(1.5 * torch.randint(-1, 2, v.shape, generator=gen))
        elif leaf == "router":
            v.zero_()
            v[:, :n] = torch.eye(n)[torch.randperm(n, generator=gen)
                                    [:v.shape[0]]]
