"""Small Nelovik configurations and weights for the tests."""

import torch


def left(heads=4, kv=2, dim=12, vdim=10, rot=6, size=11, pool=4, cap=6.0,
         scale=0.3, base=500.0):
    return {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim,
            "scale": scale, "softcap": cap,
            "rot": {"base": base, "dims": rot},
            "mask": {"size": size, "pool": pool}}


def right(heads=6, vdim=10, state=12, groups=2, conv=3, parts=3):
    return {"heads": heads, "vdim": vdim, "state": state, "groups": groups,
            "conv": conv, "norm_groups": parts}


def parallel(lft=None, rgt=None):
    return {"left": lft or left(), "right": rgt or right()}


def delta(heads=4, kv=2, dim=12, vdim=20, conv=4):
    return {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim,
            "conv": conv}


def layer(mixer, ff=None, kind=None):
    return {"type": kind or ("parallel" if "left" in mixer else "delta"),
            "mixer": mixer,
            "mlp": None if ff is None else {"kind": "dense", "ff": ff}}


def config(layers, vocab=83, width=44, eps=1e-4):
    return {"architecture": "Nelovik", "layers": layers, "vocab": vocab,
            "width": width, "norm": {"eps": eps}}


# name -> configuration; together they take every branch and unequal sizes,
# also sizes of one
CONFIGS = {
    "mixed": lambda: config([
        layer(parallel(), 30),
        layer(delta(), 24),
        layer(delta(3, 1, 17, 9, 2), None, "delta_2"),
        layer(parallel(left(3, 3, 8, 14, 8, 7, 6, base=60.0),
                       right(4, 6, 20, 4, 5, 2))),
        layer(delta(6, 6, 10, 12, 3), 40, "delta_2")]),
    # one head, one channel, a window and blocks of one token, no convolution
    # to speak of (a channel over its root mean square is near +-1: a large eps
    # keeps it from amplifying)
    "ones": lambda: config([
        layer(delta(1, 1, 1, 1, 1), 1),
        layer(parallel(left(1, 1, 2, 1, 2, 1, 1, 30.0),
                       right(1, 1, 1, 1, 1, 1)), 9),
        layer(delta(2, 2, 2, 3, 1), 5)],
        vocab=130, width=70, eps=0.05),
    # sizes without padding
    "aligned": lambda: config([
        layer(delta(4, 2, 64, 128, 4), 96),
        layer(parallel(left(8, 2, 32, 64, 16, 32, 16, 20.0),
                       right(4, 64, 128, 2, 4, 2)), 64),
        layer(delta(2, 2, 96, 32, 2), 128),
        layer(parallel(left(4, 4, 64, 32, 64, 48, 5, 50.0, 0.125),
                       right(8, 32, 32, 1, 3, 4)))],
        vocab=96, width=64, eps=1e-6),
    # large heads, norms in parts that cut heads, a long convolution, blocks
    # longer than the window
    "windows": lambda: config([
        layer(parallel(left(3, 3, 40, 70, 40, 9, 21),
                       right(5, 33, 70, 5, 8, 11)), 31),
        layer(delta(5, 1, 130, 150, 5)),
        layer(parallel(left(2, 1, 130, 9, 4, 40, 3),
                       right(2, 130, 9, 2, 2, 4)), 33)],
        vocab=64, width=32, eps=1e-5),
}


def attention_shapes(m, w):
    h, g, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    out = {"q": (h * d, w), "k": (g * d, w), "v": (g * dv, w),
           "o": (w, h * dv), "q.norm": (h * d,), "k.norm": (g * d,),
           "sink": (h,)}
    out.update({k + ".b": (out[k][0],) for k in "qkv"})
    return out


def delta_shapes(m, w):
    qk, v = m["kv_heads"] * m["dim"], m["heads"] * m["vdim"]
    out = {"q": (qk, w), "k": (qk, w), "v": (v, w), "g": (v, w),
           "a": (m["heads"], w), "b": (m["heads"], w), "o": (w, v),
           "A_log": (m["heads"],), "dt_bias": (m["heads"],),
           "norm": (m["vdim"],)}
    out.update({k + ".conv": (out[k][0], m["conv"]) for k in "qkv"})
    return out


def state_shapes(m, w):
    inner, gn = m["heads"] * m["vdim"], m["groups"] * m["state"]
    c = inner + 2 * gn
    return {"in": (inner + c + m["heads"], w), "conv": (c, m["conv"]),
            "conv.b": (c,), "dt_bias": (m["heads"],), "A_log": (m["heads"],),
            "D": (m["heads"],), "norm": (inner,), "o": (w, inner)}


def parallel_shapes(m, w):
    out = {"left." + k: s for k, s in attention_shapes(m["left"], w).items()}
    out.update({"right." + k: s for k, s in
                state_shapes(m["right"], w).items()})
    out.update({"left.out": (w,), "right.out": (w,)})
    return out


def mixer_shapes(m, w):
    return parallel_shapes(m, w) if "left" in m else delta_shapes(m, w)


def shapes(cfg):
    """checkpoint tensor names and shapes, from the configuration alone"""
    w = cfg["width"]
    out = {"embed": (cfg["vocab"], w), "head": (cfg["vocab"], w),
           "final.norm": (w,)}
    for n, lay in enumerate(cfg["layers"]):
        p = "l{}.".format(n)
        out.update({p + "mix." + k: s for k, s in
                    mixer_shapes(lay["mixer"], w).items()})
        out[p + "norm1"] = (w,)
        if lay["mlp"]:
            ff = lay["mlp"]["ff"]
            out.update({p + "norm2": (w,), p + "mlp.up": (ff, w),
                        p + "mlp.down": (w, ff), p + "mlp.act": (2,)})
    return out


def random_tensor(name, s, gen, sharp=2.5):
    """queries and keys strong enough (``sharp``) that single keys stand out;
    what is added or weighs something is neither small nor alike"""
    t = torch.randn(s, generator=gen)
    leaf = name.split(".")[-1]
    if leaf in ("norm", "norm1", "norm2", "out", "D"):
        return 1.0 + 0.3 * t
    if leaf == "A_log":  # some heads forget at once, some hardly
        return 1.5 * t - 0.5
    if leaf == "dt_bias":
        return t - 1.0
    if leaf == "embed":
        return t
    if leaf == "conv":
        return t * s[-1] ** -0.5
    if name.endswith("q.norm"):
        return sharp * t
    if len(s) == 1:
        return 0.5 * t
    return t * s[-1] ** -0.5


def weights(cfg, seed=0, sharp=2.5):
    gen = torch.Generator().manual_seed(seed)
    return {k: random_tensor(k, s, gen, sharp).to(torch.bfloat16)
            for k, s in shapes(cfg).items()}
