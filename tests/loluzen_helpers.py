"""Small random Loluzen models for the tests: ``config.json`` dictionaries and weights under their checkpoint names.

The weights are made so that every mechanism moves the logits: sharp attention scores, distance biases of a score's size,
mixing matrices with large entries beside the diagonal and of both signs, forget gates from a few tokens to hundreds, lower
bounds from zero to nearly one."""

import torch


def attention(heads, kv_heads, dim, vdim, conv, rot=None, mlp=40, scale=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": 2.5 * dim ** -0.5 if scale is None else scale, "conv": conv}
    if rot is not None:
        m["rot"] = rot
    return {"type": "attention", "mixer": m, "mlp": None if mlp is None else {"kind": "dense", "ff": mlp}}


def rot(base, dims, factor=None, low=1.0, high=4.0, original=64):
    r = {"base": base, "dims": dims}
    if factor is not None:
        r["scaling"] = {"factor": factor, "low": low, "high": high, "original": original}
    return r


def parallel(left, right, mlp=40, scale=None):
    """``left`` (heads, kv heads, dim, vdim), ``right`` (heads, dim, vdim)."""
    m = dict(zip(("heads", "kv_heads", "dim", "vdim"), left))
    m["scale"] = 2.5 * m["dim"] ** -0.5 if scale is None else scale
    return {"type": "parallel", "mixer": {"left": m, "right": dict(zip(("heads", "dim", "vdim"), right))},
            "mlp": None if mlp is None else {"kind": "dense", "ff": mlp}}


def config(width, vocab, layers, loop=None, mult=1.0, embed=1.0, eps=1e-5):
    cfg = {"architecture": "Loluzen", "width": width, "vocab": vocab, "norm": {"eps": eps}, "layers": layers, "residual_mult": mult,
           "embedding": {"scale": embed}}
    if loop is not None:
        cfg["loop"] = dict(zip(("start", "stop", "times"), loop))
    return cfg


# name -> config; sizes that differ from each other everywhere, including ones that are not multiples of 8
CONFIGS = {
    "llz-plain": config(96, 101, [parallel((4, 2, 32, 24), (3, 16, 40), 56), attention(4, 2, 24, 40, 3, rot(500.0, 16, 3.0)),
                                  parallel((4, 2, 32, 24), (3, 16, 40), None)], loop=(0, 2, 3), mult=1.2, embed=0.6),
    "llz-odd": config(76, 131, [attention(3, 1, 20, 36, 1, None, 52), parallel((6, 3, 20, 28), (5, 18, 22), 44),
                                attention(5, 5, 26, 10, 5, rot(40.0, 10, 8.0, 0.5, 2.0, 30), None), parallel((5, 1, 13, 44), (2, 44, 12), 30)],
                      loop=(3, 4, 2), mult=1.3, embed=0.5, eps=1e-3),
    "llz-wide": config(128, 64, [parallel((20, 4, 72, 136), (2, 136, 144), 72), attention(2, 1, 136, 72, 2, rot(1000.0, 136))], mult=0.9),
    "llz-heads": config(64, 50, [parallel((24, 8, 64, 32), (4, 64, 64), 48), parallel((34, 34, 8, 16), (1, 8, 72), 24), attention(8, 2, 16, 8, 4, rot(90.0, 2))],
                        loop=(1, 3, 2), mult=0.7, embed=1.5),
}


def weights(cfg, seed=0):
    g = torch.Generator().manual_seed(seed)
    w = {}
    rnd = lambda *shape: torch.randn(*shape, generator=g)

    def put(name, *shape, std=None, mean=0.0):
        std = shape[-1] ** -0.5 if std is None else std
        w[name] = (rnd(*shape) * std + mean).to(torch.bfloat16)

    width = cfg["width"]
    put("embed", cfg["vocab"], width, std=1.0)
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        for name in ("norm1", "norm1b") + (("norm2", "norm2b") if layer["mlp"] else ()):
            put(p + name, width, std=0.2)
        if layer["type"] == "attention":
            for name, rows in (("q", m["heads"] * m["dim"]), ("k", m["kv_heads"] * m["dim"]), ("v", m["kv_heads"] * m["vdim"])):
                put(f"{p}mix.{name}", rows, width)
                if m["conv"]:
                    put(f"{p}mix.{name}.conv", rows, m["conv"], std=0.6)
            for name in ("q.norm", "k.norm"):
                put(f"{p}mix.{name}", m["dim"], std=0.2, mean=1.0)
            put(p + "mix.g", m["heads"], width)
            put(p + "mix.o", width, m["heads"] * m["vdim"])
        else:
            a, r = m["left"], m["right"]
            for name, rows in (("q", a["heads"] * a["dim"]), ("k", a["kv_heads"] * a["dim"]), ("v", a["kv_heads"] * a["vdim"])):
                put(f"{p}mix.left.{name}", rows, width)
                put(f"{p}mix.left.{name}.b", rows, std=0.4)
            w[p + "mix.left.r1"] = (0.05 + 1.5 * torch.rand(a["heads"], generator=g)).to(torch.bfloat16)
            w[p + "mix.left.r2"] = (0.05 + 0.6 * torch.rand(a["heads"], generator=g)).to(torch.bfloat16)
            w[p + "mix.left.talk"] = (torch.eye(a["heads"]) + 0.9 * a["heads"] ** -0.5 * rnd(a["heads"], a["heads"])).to(torch.bfloat16)
            put(p + "mix.left.g", a["heads"], width)
            put(p + "mix.left.o", width, a["heads"] * a["vdim"])
            qk = r["heads"] * r["dim"]
            for name, rows in (("q", qk), ("f", qk), ("v", r["heads"] * r["vdim"])):
                put(f"{p}mix.right.{name}", rows, width)
            w[p + "mix.right.f.b"] = torch.linspace(-1.0, 7.0, qk).to(torch.bfloat16)
            w[p + "mix.right.lower"] = (torch.rand(qk, generator=g) * torch.linspace(0.0, 0.95, qk)).to(torch.bfloat16)
            put(p + "mix.right.norm", r["vdim"], std=0.2, mean=1.0)
            put(p + "mix.right.o", width, r["heads"] * r["vdim"])
            for side in ("left", "right"):
                put(f"{p}mix.{side}.out", width, std=0.2, mean=1.0)
        if layer["mlp"]:
            ff = layer["mlp"]["ff"]
            put(p + "mlp.up", ff, width)
            put(p + "mlp.up.b", ff, std=0.4)
            put(p + "mlp.down", width, ff)
            put(p + "mlp.down.b", width, std=0.4)
    put("final.norm", width, std=0.2)
    put("head", cfg["vocab"], width, std=1.5 * width ** -0.5)
    return w
