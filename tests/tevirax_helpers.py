"""Small random Tevirax models for the tests: ``config.json`` dictionaries and weights under their checkpoint names.

The weights are made so that every mechanism moves the logits: sharp attention scores, forget gates that keep for tens of
tokens, step sizes over two orders of magnitude.  The choice of experts must not rest on a close call (a bf16 rounding
would turn it), so the last columns of the residual are left alone by every layer (norm weights of zero) and carry, per
token, the router's logits as a permutation of separated levels; the other columns only add to them a little."""

import math

import torch


def mamba2(heads, vdim, state, groups, conv, norm_groups, mlp):
    return {"type": "mamba2", "mlp": mlp, "mixer": {"heads": heads, "vdim": vdim, "state": state, "groups": groups, "conv": conv,
                                                    "norm_groups": norm_groups}}


def parallel(left, right, mlp, left_scale=0.8, right_scale=1.3):
    return {"type": "parallel", "mlp": mlp, "mixer": {"left": left, "right": right, "left_scale": left_scale, "right_scale": right_scale}}


def left(heads, kv_heads, dim, vdim, chunk, rot_dims, base=700.0, scaling=(2.0, 40, 8.0, 1.0), scale=None):
    d = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": 1.7 * dim ** -0.5 if scale is None else scale,
         "mask": {"size": chunk}, "rot": {"base": base, "dims": rot_dims}}
    if scaling is not None:
        d["rot"]["scaling"] = dict(zip(("factor", "original", "fast", "slow"), scaling))
    return d


def right(heads, dim, vdim, cap=9.0):
    return {"heads": heads, "dim": dim, "vdim": vdim, "gate_cap": cap}


def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(experts, ff, top, groups=None, shared=None):
    router = {"experts": experts, "top": top}
    if groups is not None:
        router["groups"] = {"count": groups[0], "keep": groups[1]}
    d = {"kind": "moe", "expert": {"ff": ff}, "router": router}
    if shared is not None:
        d["shared"] = {"ff": shared}
    return d


def config(width, vocab, layers, eps=1e-5, scale=6.0, positions=700, cap=20.0):
    return {"architecture": "Tevirax", "width": width, "vocab": vocab, "norm": {"eps": eps}, "layers": layers,
            "embedding": {"scale": scale}, "logit_softcap": cap, "max_positions": positions}


# name -> config; sizes that differ from each other everywhere, including ones that are not multiples of 8
CONFIGS = {
    "tvx-plain": config(88, 101, [mamba2(3, 16, 24, 1, 4, 1, dense(40)),
                                  parallel(left(4, 2, 32, 24, 19, 12), right(3, 24, 40), moe(6, 24, 2, (3, 2), 40)),
                                  mamba2(4, 24, 40, 2, 3, 4, moe(8, 40, 3, None, 24))], cap=4.0),
    "tvx-odd": config(76, 131, [parallel(left(6, 3, 20, 36, 7, 10, scaling=None), right(2, 12, 20, 3.0), None, 1.4, 0.5),
                                mamba2(6, 20, 18, 3, 1, 3, moe(5, 22, 4, None, None)),
                                parallel(left(3, 1, 44, 28, 33, 44, 50.0, (3.0, 24, 4.0, 0.5)), right(5, 30, 14), dense(28)),
                                mamba2(2, 44, 33, 1, 6, 2, None)], eps=1e-3, scale=3.0, cap=7.0),
    "tvx-wide": config(128, 64, [mamba2(2, 144, 160, 2, 2, 1, dense(72)),
                                 parallel(left(4, 2, 48, 320, 40, 48, 1000.0, (4.0, 64, 16.0, 1.0)), right(2, 136, 200), moe(12, 72, 4, (4, 3), 56)),
                                 parallel(left(8, 2, 136, 72, 70, 40), right(1, 72, 136, 14.0), dense(40))]),
}


def levels(experts):
    """Router logits of a token, in some order.  Their scores fall by a constant factor, so that no two sums of two scores
    come close."""
    scores = [0.93 * 0.6 ** e for e in range(experts)]
    return [math.log(s / (1 - s)) for s in scores]


def weights(cfg, seed=0):
    g = torch.Generator().manual_seed(seed)
    w = {}
    rnd = lambda *shape: torch.randn(*shape, generator=g)

    def put(name, *shape, std=None, mean=0.0):
        std = shape[-1] ** -0.5 if std is None else std
        w[name] = (rnd(*shape) * std + mean).to(torch.bfloat16)

    width, vocab = cfg["width"], cfg["vocab"]
    experts = max([l["mlp"]["router"]["experts"] for l in cfg["layers"] if l["mlp"] and l["mlp"]["kind"] == "moe"], default=0)
    free = width - experts  # columns that layers write

    def norm(name, std=0.2):
        put(name, width, std=std, mean=1.0)
        w[name][free:] = 0

    def mlp(p, ff):
        put(p + "gate", ff, width)
        put(p + "up", ff, width)
        put(p + "down", width, ff)

    put("embed", vocab, width, std=1.0 / cfg["embedding"]["scale"])
    put("pos", cfg["max_positions"], width, std=0.5)
    lv = torch.tensor(levels(experts))
    for t in range(vocab):
        w["embed"][t, free:] = (2.0 * lv[torch.randperm(experts, generator=g)] / cfg["embedding"]["scale"]).to(torch.bfloat16)
    w["pos"][:, free:] = 0
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        norm(p + "norm1")
        if layer["type"] == "mamba2":
            inner, gn, heads = m["heads"] * m["vdim"], m["groups"] * m["state"], m["heads"]
            put(p + "mix.in", 2 * inner + 2 * gn + heads, width, std=0.5 * width ** -0.5)
            put(p + "mix.conv", inner + 2 * gn, m["conv"], std=0.7)
            put(p + "mix.conv.b", inner + 2 * gn, std=0.3)
            w[p + "mix.dt_bias"] = torch.linspace(-4.0, 0.5, heads).to(torch.bfloat16)
            w[p + "mix.A_log"] = (rnd(heads) * 0.7).to(torch.bfloat16)
            put(p + "mix.D", heads, std=0.5, mean=1.0)
            put(p + "mix.norm", inner, std=0.2, mean=1.0)
            put(p + "mix.o", width, inner)
        else:
            a, r = m["left"], m["right"]
            for n, rows in (("q", a["heads"] * a["dim"]), ("k", a["kv_heads"] * a["dim"]), ("v", a["kv_heads"] * a["vdim"])):
                put(f"{p}mix.left.{n}", rows, width)
            put(p + "mix.left.q.norm", a["dim"], std=0.3, mean=1.2)
            put(p + "mix.left.k.norm", a["dim"], std=0.3, mean=1.2)
            put(p + "mix.left.o", width, a["heads"] * a["vdim"])
            inner = r["heads"] * r["vdim"]
            for n, rows in (("q", r["heads"] * r["dim"]), ("k", r["heads"] * r["dim"]), ("v", inner), ("g", inner)):
                put(f"{p}mix.right.{n}", rows, width, std=0.6 * width ** -0.5)
            for n, mean in (("i", -1.0), ("f", 3.5)):
                put(f"{p}mix.right.{n}", r["heads"], width, std=0.7 * width ** -0.5)
                put(f"{p}mix.right.{n}.b", r["heads"], std=1.0, mean=mean)
            put(p + "mix.right.norm", inner, std=0.2, mean=1.0)
            put(p + "mix.right.o", width, inner)
        ff = layer["mlp"]
        if ff is None:
            continue
        norm(p + "norm2")
        if ff["kind"] == "dense":
            mlp(p + "mlp.", ff["ff"])
            continue
        n = ff["router"]["experts"]
        router = 0.003 * rnd(n, width)
        router[:, free:] = 0.5 * torch.eye(n, experts)
        w[p + "mlp.router"] = router.to(torch.bfloat16)
        for e in range(n):
            mlp(f"{p}mlp.e{e}.", ff["expert"]["ff"])
        if ff.get("shared"):
            mlp(p + "mlp.shared.", ff["shared"]["ff"])
            put(p + "mlp.shared.sg", 1, width)
    put("final.norm", width, std=0.2, mean=1.0)
    put("head", vocab, width, std=1.5 * width ** -0.5)
    return w
