"""Small Kakipel configurations and weights for the tests."""

import torch


def yarn(factor=3.0, original=40, fast=8.0, slow=0.5):
    return {"factor": factor, "original": original, "fast": fast,
            "slow": slow}


def attn(heads=3, dim=12, rot=6, vdim=10, q_rank=14, rank=20, base=500.0,
         scale=0.3, scaling=True):
    out = {"heads": heads, "dim": dim, "rot_dim": rot, "vdim": vdim,
           "q_rank": q_rank, "kv_rank": rank, "scale": scale,
           "rot": {"base": base, "dims": rot}}
    if scaling:
        out["rot"]["scaling"] = yarn() if scaling is True else scaling
    return out


def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(experts, top, ff):
    return {"kind": "moe", "expert": {"ff": ff},
            "router": {"experts": experts, "top": top}}


def layer(mixer, mlp=None):
    return {"type": "latent_attention", "mixer": mixer, "mlp": mlp}


def config(layers, loop=None, vocab=83, width=44, eps=1e-4):
    out = {"architecture": "Kakipel", "layers": layers, "vocab": vocab,
           "width": width, "norm": {"eps": eps}}
    if loop is not None:
        out["loop"] = dict(zip(("start", "stop", "times"), loop))
    return out


# name -> configuration; together they take every branch and unequal sizes,
# also sizes of one
CONFIGS = {
    # the loop lies inside, one of its layers has no feed-forward
    "mixed": lambda: config([
        layer(attn(), dense(36)),
        layer(attn(heads=2, dim=8, rot=10, vdim=14, q_rank=33, rank=9,
                   scale=0.45), moe(5, 2, 24)),
        layer(attn(heads=5, vdim=3, scaling=yarn(8.0, 16, 4.0, 2.0))),
        layer(attn(rot=2, base=77.0), moe(3, 1, 40))], loop=(1, 3, 2)),
    # everything is looped; one head, a latent of one, every expert chosen
    # (a latent of one is near +-1: a large eps keeps it from amplifying)
    "all_looped": lambda: config([
        layer(attn(heads=1, dim=40, rot=34, vdim=36, q_rank=1, rank=70,
                   scaling=False), moe(7, 7, 1)),
        layer(attn(heads=17, dim=1, rot=4, vdim=1, q_rank=40, rank=1,
                   scale=1.0), dense(1))],
        loop=(0, 2, 3), vocab=130, width=70, eps=0.05),
    # nothing is; sizes that the tiled expert products take
    "no_loop": lambda: config([
        layer(attn(heads=4, dim=32, rot=32, vdim=32, q_rank=96, rank=64),
              moe(6, 3, 64)),
        layer(attn(heads=2, dim=64, rot=16, vdim=48, q_rank=32, rank=96),
              moe(9, 2, 128))], vocab=96, width=64, eps=1e-6),
    # the loop ends the model and runs once
    "ends_in_loop": lambda: config([
        layer(attn(), moe(1, 1, 30)),
        layer(attn(heads=4, dim=6, rot=6, q_rank=70, rank=33)),
        layer(attn(heads=2), dense(50))],
        loop=(2, 3, 1), vocab=64, width=32),
}


def runs(cfg):
    """number of layer runs"""
    loop = cfg.get("loop")
    extra = 0 if loop is None else \
        (loop["stop"] - loop["start"]) * (loop["times"] - 1)
    return len(cfg["layers"]) + extra


def shapes(cfg):
    """checkpoint tensor names and shapes, from the configuration alone"""
    w = cfg["width"]
    out = {"embed": (cfg["vocab"], w), "head": (cfg["vocab"], w),
           "final.norm": (w,)}
    if "loop" in cfg:
        out["loop.in"] = (w, 2 * w)
        out["loop.step"] = (cfg["loop"]["times"], w)
    for n, lay in enumerate(cfg["layers"]):
        m, p, f = lay["mixer"], "l{}.".format(n), lay["mlp"]
        h, dr = m["heads"], m["dim"] + m["rot_dim"]
        mix = {"dq": (m["q_rank"], w), "dq.norm": (m["q_rank"],),
               "uq": (h * dr, m["q_rank"]),
               "dkv": (m["kv_rank"] + m["rot_dim"], w),
               "dkv.norm": (m["kv_rank"],),
               "uk": (h * m["dim"], m["kv_rank"]),
               "uv": (h * m["vdim"], m["kv_rank"]),
               "g": (h * m["vdim"], w), "o": (w, h * m["vdim"])}
        out.update({p + "mix." + k: s for k, s in mix.items()})
        for k in ("norm1", "norm1b") + (("norm2", "norm2b") if f else ()):
            out[p + k] = (w,)
        if f is None:
            continue
        if f["kind"] == "dense":
            mlp = {"gate": (f["ff"], w), "up": (f["ff"], w),
                   "down": (w, f["ff"])}
        else:
            e = f["expert"]["ff"]
            mlp = {"router": (f["router"]["experts"], w)}
            for k in range(f["router"]["experts"]):
                mlp["e{}.up".format(k)] = (e, w)
                mlp["e{}.down".format(k)] = (w, e)
        out.update({p + "mlp." + k: s for k, s in mlp.items()})
    return out


def weights(cfg, seed=0, sharp=2.5, decided=False):
    """Random, with queries strong enough (``sharp``) that single keys stand
    out.

    ``decided``: no routing is a close call, whatever the rounding. A few
    stream coordinates, one per expert, are set by the token alone (sublayers
    do not touch them, passes of the loop hand them on); the routers read
    only these."""
    gen = torch.Generator().manual_seed(seed)
    out = {}
    for name, s in shapes(cfg).items():
        t = torch.randn(s, generator=gen)
        leaf = name.split(".", 2)[-1]
        if name == "embed":
            pass
        elif leaf == "uq":
            t = t * sharp * s[-1] ** -0.5
        elif len(s) == 1:  # norms
            t = 1.0 + 0.3 * t
        elif name == "loop.step":
            t = 0.5 * t
        else:
            t = t * s[-1] ** -0.5
        out[name] = t
    if decided:
        _decide(cfg, out, gen)
    return {k: v.to(torch.bfloat16) for k, v in out.items()}


def _decide(cfg, st, gen):
    n = max([lay["mlp"]["router"]["experts"] for lay in cfg["layers"]
             if lay["mlp"] and lay["mlp"]["kind"] == "moe"], default=0)
    w = cfg["width"]
    assert 0 < n <= w // 3
    # distances of 1.5 between the levels a token gives the experts
    levels = 1.5 * (torch.arange(n) - (n - 1) / 2)
    for v in range(cfg["vocab"]):
        st["embed"][v, :n] = levels[torch.randperm(n, generator=gen)]
    if "loop" in cfg:
        st["loop.in"][:n] = 0
        st["loop.in"][:n, w:w + n] = torch.eye(n)
        st["loop.step"][:, :n] = 0
    for i, lay in enumerate(cfg["layers"]):
        p = "l{}.".format(i)
        for k in ("norm1b", "norm2b"):
            if p + k in st:
                st[p + k][:n] = 0
        if p + "mlp.router" in st:
            r = st[p + "mlp.router"]
            e = r.shape[0]
            st[p + "norm2"][:n] = 1.0
            r.zero_()
            r[:, :n] = torch.eye(n)[torch.randperm(n, generator=gen)[:e]]
