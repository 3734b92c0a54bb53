"""Small random Vusalix models for the tests: ``config.json`` dictionaries and weights under their checkpoint names.

The weights are made so that every mechanism moves the logits: sharp attention scores, biases and sinks of a score's size,
decays from a few tokens to hundreds.  The choice of experts must not rest on a close call (a bf16 rounding would turn it),
so the last columns of the residual are written by no projection and carry, per token, the router's logits as a permutation
of separated levels (identity experts and the mixing of streams only scale them); the other columns add a little."""

import torch


def delta(heads, kv_heads, dim, vdim, conv, mlp):
    return {"type": "delta", "mlp": mlp, "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv}}


def latent(heads, dim, rot_dim, vdim, kv_rank, window, mlp, base=900.0, scaling=(3.0, 60, 8.0, 1.0), scale=None):
    m = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank, "mask": {"size": window},
         "scale": 2.0 * (dim + rot_dim) ** -0.5 if scale is None else scale, "rot": {"base": base, "dims": rot_dim}}
    if scaling is not None:
        m["rot"]["scaling"] = dict(zip(("factor", "original", "fast", "slow"), scaling))
    return {"type": "latent_attention", "mlp": mlp, "mixer": m}


def attention(heads, kv_heads, dim, vdim, window, bias_max, softcap, mlp, scale=None, buckets=12):
    return {"type": "attention", "mlp": mlp, "buckets": buckets,
            "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "mask": {"size": window}, "bias_max": bias_max,
                      "softcap": softcap, "scale": 2.0 * dim ** -0.5 if scale is None else scale}}


def moe(experts, ff, top, identity=0, groups=None, shared=None):
    router = {"experts": experts, "top": top, "identity": identity}
    if groups is not None:
        router["groups"] = {"count": groups[0], "keep": groups[1]}
    d = {"kind": "moe", "expert": {"ff": ff}, "router": router}
    if shared is not None:
        d["shared"] = {"ff": shared}
    return d


def config(width, vocab, layers, streams, eps=1e-5):
    """``layers`` as the functions above make them; a table's length is not part of a ``config.json``."""
    cfg = {"architecture": "Vusalix", "width": width, "vocab": vocab, "norm": {"eps": eps}, "streams": streams,
           "layers": [{k: v for k, v in layer.items() if k != "buckets"} for layer in layers]}
    BUCKETS[id(cfg)] = [layer.get("buckets") for layer in layers]
    return cfg


BUCKETS = {}

# name -> config; sizes that differ from each other everywhere, including ones that are not multiples of 8
CONFIGS = {
    "vsx-plain": config(96, 101, [delta(4, 2, 32, 24, 4, moe(6, 24, 2, 2, (2, 1), 40)),
                                  latent(3, 24, 8, 40, 56, 21, moe(5, 32, 3, 3, (4, 3), 24)),
                                  attention(4, 2, 32, 24, 37, 30, 9.0, moe(7, 24, 2, 1, None, 56))], 2),
    "vsx-odd": config(76, 131, [attention(6, 2, 20, 36, 7, 11, 4.0, None, buckets=6), latent(2, 13, 6, 21, 27, 33, moe(5, 22, 4), scaling=None, base=40.0),
                                delta(6, 3, 18, 22, 1, moe(6, 30, 1, 3, (3, 2), None)), delta(3, 1, 44, 28, 2, None),
                                attention(3, 1, 44, 28, 64, 200, 25.0, moe(4, 26, 3, 4, (2, 2), 18), buckets=4)], 5, eps=1e-3),
    "vsx-wide": config(128, 64, [latent(5, 136, 24, 72, 200, 40, moe(8, 72, 4, 4, (4, 3), 56)), attention(8, 2, 136, 200, 70, 64, 15.0, None),
                                 delta(2, 2, 144, 160, 3, moe(3, 40, 2)), latent(20, 16, 8, 32, 24, None, None, base=50.0)], 1),
}


def router_width(cfg):
    return max([l["mlp"]["router"]["experts"] + l["mlp"]["router"]["identity"] for l in cfg["layers"] if l["mlp"]], default=0)


def weights(cfg, seed=0):
    g = torch.Generator().manual_seed(seed)
    w = {}
    rnd = lambda *shape: torch.randn(*shape, generator=g)

    def put(name, *shape, std=None, mean=0.0):
        std = shape[-1] ** -0.5 if std is None else std
        w[name] = (rnd(*shape) * std + mean).to(torch.bfloat16)

    width, vocab, levels = cfg["width"], cfg["vocab"], router_width(cfg)
    free = width - levels  # columns that projections write

    def back(name, inner, std=None):
        put(name, width, inner, std=std)
        w[name][free:] = 0

    def norm(name):
        put(name, width, std=0.2, mean=1.0)
        w[name][free:] = 1

    def mlp(p, ff):
        put(p + "gate", ff, width)
        put(p + "up", ff, width)
        back(p + "down", ff, std=2.0 * ff ** -0.5)

    put("embed", vocab, width, std=1.0)
    lv = torch.linspace(-1.5, 1.5, levels) if levels else torch.empty(0)
    for t in range(vocab):
        w["embed"][t, free:] = lv[torch.randperm(levels, generator=g)].to(torch.bfloat16)
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        norm(p + "norm1")
        n = cfg["streams"]
        for hc in ("hc1.", "hc2.")[: 1 + (layer["mlp"] is not None)]:
            put(p + hc + "in", n, std=0.2 / n, mean=1.0 / n)
            put(p + hc + "out", n, std=0.3, mean=0.7)
            w[p + hc + "mix"] = (torch.eye(n) * 0.7 + 0.3 / n + 0.1 / n * rnd(n, n)).to(torch.bfloat16)
        if layer["type"] == "delta":
            heads, inner = m["heads"], m["heads"] * m["vdim"]
            for name, rows in (("q", m["kv_heads"] * m["dim"]), ("k", m["kv_heads"] * m["dim"]), ("v", inner)):
                put(f"{p}mix.{name}", rows, width)
                put(f"{p}mix.{name}.conv", rows, m["conv"], std=0.6)
            put(p + "mix.b", heads, width)
            put(p + "mix.a", heads, width, std=0.5 * width ** -0.5)
            put(p + "mix.g", inner, width)
            w[p + "mix.A_log"] = (rnd(heads) * 0.5).to(torch.bfloat16)
            w[p + "mix.dt_bias"] = torch.linspace(-5.0, -1.0, heads).to(torch.bfloat16)
            put(p + "mix.norm", m["vdim"], std=0.2, mean=1.0)
            back(p + "mix.o", inner)
        elif layer["type"] == "latent_attention":
            put(p + "mix.q", m["heads"] * (m["dim"] + m["rot_dim"]), width)
            put(p + "mix.dkv", m["kv_rank"] + m["rot_dim"], width)
            put(p + "mix.dkv.norm", m["kv_rank"], std=0.2, mean=1.0)
            put(p + "mix.uk", m["heads"] * m["dim"], m["kv_rank"])
            put(p + "mix.uv", m["heads"] * m["vdim"], m["kv_rank"])
            back(p + "mix.o", m["heads"] * m["vdim"])
        else:
            for name, rows in (("q", m["heads"] * m["dim"]), ("k", m["kv_heads"] * m["dim"]), ("v", m["kv_heads"] * m["vdim"])):
                put(f"{p}mix.{name}", rows, width)
            put(p + "mix.rel", BUCKETS[id(cfg)][i], m["heads"], std=1.0)
            put(p + "mix.sink", m["heads"], std=1.0)
            back(p + "mix.o", m["heads"] * m["vdim"])
        ff = layer["mlp"]
        if ff is None:
            continue
        norm(p + "norm2")
        every = ff["router"]["experts"] + ff["router"]["identity"]
        router = 0.003 * rnd(every, width)
        router[:, free:] = 2.0 * torch.eye(every, levels)
        w[p + "mlp.router"] = router.to(torch.bfloat16)
        # some experts preferred by much more than scores differ, the rest not at all
        w[p + "mlp.correction"] = torch.where(rnd(every) > 0.8, 2.0, 0.0).to(torch.bfloat16)
        for e in range(ff["router"]["experts"]):
            mlp(f"{p}mlp.e{e}.", ff["expert"]["ff"])
        if ff.get("shared"):
            mlp(p + "mlp.shared.", ff["shared"]["ff"])
    put("final.norm", width, std=0.2, mean=1.0)
    put("head", vocab, width, std=1.5 * width ** -0.5)
    return w
