"""Small random hybrid models for the tests: a ``config.json`` dictionary, weights under their checkpoint names, a
checkpoint folder of both, and the oracle of the design (Lotozen here, Tevirax in tevirax_helpers.py, Vusalix in
vusalix_helpers.py, Loluzen in loluzen_helpers.py)."""

import json
import os

import numpy as np
import torch

from oracle import hybrid_oracle, loluzen_oracle, tevirax_oracle, vusalix_oracle
from tests import loluzen_helpers as lz, tevirax_helpers as tv, vusalix_helpers as vx


def attention(heads, kv_heads, dim, vdim, window, conv, rot_dims, base=1000.0, factor=1.0, scale=None, v_mix=True, ff=40):
    return {"type": "attention", "mlp": None if ff is None else {"kind": "dense", "ff": ff},
            "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv, "v_mix": v_mix,
                      "scale": 2.5 * dim ** -0.5 if scale is None else scale, "mask": {"size": window},
                      "rot": {"base": base, "dims": rot_dims, "scaling": {"factor": factor}}}}


def lightning(heads, dim, vdim, decay, ff=40):
    return {"type": "lightning", "mlp": None if ff is None else {"kind": "dense", "ff": ff},
            "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "decay": list(decay)}}


def config(width, vocab, layers, eps=1e-5, side=None):
    cfg = {"architecture": "Lotozen", "width": width, "vocab": vocab, "norm": {"eps": eps}, "layers": layers}
    if side is not None:
        cfg["token_side"] = {"dim": side}
    return cfg


# name -> config; sizes that differ from each other everywhere, including ones that are not multiples of 8
CONFIGS = {
    "plain": config(64, 97, [attention(4, 2, 32, 24, 19, 4, 12, factor=2.0), lightning(3, 16, 32, [0.7, 0.98, 0.9995]),
                             attention(4, 2, 32, 24, 19, 4, 12, factor=2.0)], side=8),
    "odd": config(76, 131, [lightning(2, 36, 20, [0.9, 0.99], ff=52), attention(6, 3, 20, 36, 7, 2, 10, v_mix=False, ff=None),
                            attention(3, 1, 44, 36, 33, 5, 44, base=50.0, factor=3.0, ff=28),
                            lightning(5, 24, 16, [0.0, 0.5, 0.9, 0.99, 1.0], ff=None),
                            attention(5, 1, 28, 36, 40, 1, 2, ff=30)], eps=1e-3, side=5),
    "wide-heads": config(128, 64, [attention(2, 2, 64, 160, 70, 3, 64), attention(8, 2, 136, 160, 16, 6, 40, factor=1.5),
                                   lightning(2, 96, 144, [0.95, 0.999])]),
    "no-mixing": config(48, 50, [attention(4, 4, 16, 16, 1, 3, 16, v_mix=False), attention(4, 1, 24, 8, 300, 8, 8, v_mix=False),
                                 lightning(1, 8, 8, [0.97])], side=3),
}


CONFIGS.update(tv.CONFIGS)
CONFIGS.update(vx.CONFIGS)
CONFIGS.update(lz.CONFIGS)


def forward(w, cfg, tokens, **kw):
    """The oracle's logits of a whole sequence."""
    oracle = {"Lotozen": hybrid_oracle, "Tevirax": tevirax_oracle, "Vusalix": vusalix_oracle, "Loluzen": loluzen_oracle}[cfg["architecture"]]
    return oracle.decoder_forward(w, cfg, tokens, **kw)


def weights(cfg, seed=0):
    """bfloat16 tensors (as stored in a checkpoint) scaled so that every mechanism moves the logits."""
    if cfg["architecture"] == "Tevirax":
        return tv.weights(cfg, seed)
    if cfg["architecture"] == "Vusalix":
        return vx.weights(cfg, seed)
    if cfg["architecture"] == "Loluzen":
        return lz.weights(cfg, seed)
    g = torch.Generator().manual_seed(seed)
    w = {}

    def put(name, *shape, std=None, mean=0.0):
        std = shape[-1] ** -0.5 if std is None else std
        w[name] = (torch.randn(*shape, generator=g) * std + mean).to(torch.bfloat16)

    def norm(name):
        put(name, cfg["width"], std=0.2, mean=1.0)
        put(name + ".b", cfg["width"], std=0.2)

    width, side = cfg["width"], cfg.get("token_side", {}).get("dim", 0)
    put("embed", cfg["vocab"], width, std=1.0)
    if side:
        put("side.embed", cfg["vocab"], side * len(cfg["layers"]), std=1.0)
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        norm(p + "norm1")
        if layer["type"] == "attention":
            for n, rows in (("q", m["heads"] * m["dim"]), ("k", m["kv_heads"] * m["dim"]), ("v", m["kv_heads"] * m["vdim"])):
                put(f"{p}mix.{n}", rows, width)
                put(f"{p}mix.{n}.conv", rows, m["conv"], std=0.6)
            put(p + "mix.g", m["heads"], width)
            put(p + "mix.o", width, m["heads"] * m["vdim"])
            if m["v_mix"]:
                w[p + "mix.vmix"] = torch.tensor(0.3 + 0.1 * i).to(torch.bfloat16)
        else:
            inner = m["heads"] * m["vdim"]
            for n, rows in (("q", m["heads"] * m["dim"]), ("k", m["heads"] * m["dim"]), ("v", inner), ("g", inner)):
                put(f"{p}mix.{n}", rows, width)
            put(p + "mix.o", width, inner)
            put(p + "mix.norm", inner, std=0.2, mean=1.0)
        if layer["mlp"] is not None:
            ff = layer["mlp"]["ff"]
            norm(p + "norm2")
            put(p + "mlp.gate", ff, width)
            put(p + "mlp.up", ff, width)
            put(p + "mlp.down", width, ff)
        if side:
            put(p + "side.gate", side, width)
            put(p + "side.proj", width, side)
            put(p + "side.norm", width, std=0.2, mean=1.0)
    norm("final.norm")
    put("head", cfg["vocab"], width)
    return w


def save(folder, cfg, w):
    from safetensors.torch import save_file

    os.makedirs(folder, exist_ok=True)
    with open(os.path.join(folder, "config.json"), "w") as fh:
        json.dump(cfg, fh)
    save_file({k: v.contiguous() for k, v in w.items()}, os.path.join(folder, "model.safetensors"))
    return str(folder)


def prompts(cfg, lens, seed=1):
    g = np.random.default_rng(seed)
    return [g.integers(0, cfg["vocab"], n).tolist() for n in lens]


def logit_error(got, want):
    """Root mean square difference per position, means taken off, over the root mean square of the logits."""
    d = got.double() - want.double()
    d = d - d.mean(-1, keepdim=True)
    c = want.double() - want.double().mean(-1, keepdim=True)
    return d.pow(2).mean(-1).sqrt() / c.pow(2).mean().sqrt()


def bf16_tolerance(forward, cfg, w, tokens, want, runs=3):
    """Per position, what rounding to bf16 may do to the logits: four times what noise of bf16's size on every weight does
    to the oracle's, and never less than 0.03 (some positions are ill-conditioned: a normed sum that nearly cancels, two
    keys that nearly tie)."""
    g = torch.Generator().manual_seed(5)
    worst = torch.full((len(tokens),), 0.0075, dtype=torch.float64)
    for _ in range(runs):
        noisy = {n: t.double() * (1 + 2.0 ** -9 * torch.randn(t.shape, generator=g, dtype=torch.float64)) for n, t in w.items()}
        worst = torch.maximum(worst, logit_error(forward(noisy, cfg, tokens), want))
    return 4 * worst
