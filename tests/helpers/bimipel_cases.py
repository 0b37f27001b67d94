"""Small Bimipel configurations and weights for the tests."""

import torch


def attn(heads=3, dim=12, rot=6, vdim=10, rank=20, window=7, base=500.0,
         scale=0.3, kv_from=None):
    m = {"heads": heads, "dim": dim, "rot_dim": rot, "vdim": vdim,
         "kv_rank": rank, "scale": scale, "mask": {"size": window},
         "rot": {"base": base, "dims": rot}}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return m


def rec(width=24, blocks=3, conv=4):
    return {"width": width, "blocks": blocks, "conv": conv}


def layer(mixer, ff=None):
    return {"type": "rglru" if "conv" in mixer else "latent_attention",
            "mixer": mixer,
            "mlp": None if ff is None else {"kind": "dense", "ff": ff}}


def config(layers, vocab=83, width=44, eps=1e-4, logit_scale=0.7):
    return {"architecture": "Bimipel", "layers": layers, "vocab": vocab,
            "width": width, "norm": {"eps": eps}, "logit_scale": logit_scale}


# name -> configuration; together they take every branch and unequal sizes,
# also sizes of one
CONFIGS = {
    "mixed": lambda: config([
        layer(attn(window=7), ff=36),
        layer(rec(24, 3, 4)),
        layer(attn(heads=2, dim=8, vdim=14, window=19, scale=0.45,
                   kv_from=0), ff=52),
        layer(rec(20, 1, 2), ff=28)]),
    "recurrent_first": lambda: config([
        layer(rec(33, 3, 1), ff=20),
        layer(attn(heads=1, dim=40, rot=34, vdim=36, rank=70, window=33)),
        layer(rec(64, 2, 6)),
        layer(attn(heads=17, dim=4, rot=2, vdim=3, rank=9, window=1,
                   base=77.0, scale=1.0), ff=1),
        layer(attn(heads=5, dim=6, rot=34, vdim=8, rank=70, window=70,
                   kv_from=1), ff=30)],
        vocab=130, width=70, eps=1e-6, logit_scale=1.9),
    "attention_only": lambda: config([
        layer(attn(heads=4, dim=32, rot=32, vdim=32, rank=64, window=65),
              ff=64),
        layer(attn(heads=4, dim=32, rot=32, vdim=32, rank=64, window=130,
                   kv_from=0))],
        vocab=96, width=64, eps=1e-5, logit_scale=1.0),
    "recurrent_only": lambda: config(
        [layer(rec(96, 3, 4), ff=40), layer(rec(40, 5, 3))],
        vocab=64, width=32, eps=1e-5, logit_scale=0.25),
}


def shapes(cfg):
    """checkpoint tensor names and shapes, from the configuration alone"""
    w = cfg["width"]
    out = {"embed": (cfg["vocab"], w), "final.norm": (w,)}
    for n, lay in enumerate(cfg["layers"]):
        m, p = lay["mixer"], "l{}.".format(n)
        out[p + "norm1"] = (w,)
        mix = {}
        if lay["type"] == "latent_attention":
            h = m["heads"]
            mix = {"q": (h * (m["dim"] + m["rot_dim"]), w),
                   "uk": (h * m["dim"], m["kv_rank"]),
                   "uv": (h * m["vdim"], m["kv_rank"]), "sink": (h,),
                   "o": (w, h * m["vdim"])}
            if m.get("kv_from") is None:
                mix["dkv"] = (m["kv_rank"] + m["rot_dim"], w)
                mix["dkv.norm"] = (m["kv_rank"],)
        else:
            c, b = m["width"], m["blocks"]
            k = c // b
            mix = {"y": (c, w), "y.b": (c,), "x": (c, w), "x.b": (c,),
                   "conv": (c, m["conv"]), "conv.b": (c,),
                   "ra": (b, k, k), "ra.b": (b, k), "ri": (b, k, k),
                   "ri.b": (b, k), "lam": (c,), "o": (w, c)}
        for k, s in mix.items():
            out[p + "mix." + k] = s
        if lay["mlp"] is not None:
            f = lay["mlp"]["ff"]
            out[p + "norm2"] = (w,)
            for k, s in {"gate": (f, w), "gate.b": (f,), "up": (f, w),
                         "up.b": (f,), "down": (w, f),
                         "down.b": (w,)}.items():
                out[p + "mlp." + k] = s
    return out


def weights(cfg, seed=0, sharp=2.5):
    """Random, with queries strong enough (``sharp``) that single keys stand
    out, sinks of both signs and decays from short to long memory."""
    gen = torch.Generator().manual_seed(seed)
    out = {}
    for name, s in shapes(cfg).items():
        t = torch.randn(s, generator=gen)
        leaf = name.split(".", 2)[-1]
        if name == "embed":
            pass
        elif leaf == "q":
            t = t * sharp * s[-1] ** -0.5
        elif leaf == "dkv.norm":
            t = 1.0 + 0.3 * t
        elif leaf == "sink":
            t = 1.5 * t
        elif leaf == "lam":
            t = -3.0 + 2.5 * t
        elif leaf == "conv":
            t = t * 0.6
        elif len(s) == 1 or leaf.endswith(".b"):
            t = t * 0.3
        else:
            t = t * s[-1] ** -0.5
        out[name] = t.to(torch.bfloat16)
    return out
