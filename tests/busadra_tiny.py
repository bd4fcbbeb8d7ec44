"""Tiny Busadra configurations for tests, with random weights of a scale at which every mechanism moves the logits
(scores large enough for the soft cap to bend them, forget gates from near 0 to near 1, layer scales, convolutions and
depth averages away from the trivial), written as model folders.  Sizes differ from one another wherever the design
allows."""
import json
import math
import os
import random

import torch


def _moe(ff, experts, top):
    return {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}


# A: both mixers, key and value sizes that differ, grouped heads, a rotation of part of a head with all three bands of
# wavelengths, a layer without a feed-forward, two experts chosen.
BA = {
    "architecture": "Busadra", "vocab": 211, "width": 96, "norm": {"eps": 1e-6}, "canon": {"taps": 3}, "logit_scale": 0.7,
    "layers": [
        {"type": "attention",
         "mixer": {"heads": 6, "kv_heads": 2, "dim": 20, "vdim": 12, "mask": {"size": 37}, "scale": 0.4, "softcap": 4.0,
                   "rot": {"base": 500.0, "dims": 12, "scaling": {"factor": 6.0, "low": 1.0, "high": 4.0, "original": 64}}},
         "mlp": _moe(40, 6, 2)},
        {"type": "hgrn2", "mixer": {"heads": 3, "dim": 12, "vdim": 20}, "mlp": None},
        {"type": "hgrn2", "mixer": {"heads": 2, "dim": 28, "vdim": 16}, "mlp": _moe(24, 5, 3)},
        {"type": "attention",
         "mixer": {"heads": 4, "kv_heads": 4, "dim": 16, "vdim": 24, "mask": {"size": 9}, "scale": 0.3, "softcap": 15.0,
                   "rot": {"base": 1000.0, "dims": 16, "scaling": {"factor": 2.0, "low": 0.5, "high": 2.0, "original": 300}}},
         "mlp": _moe(56, 4, 1)},
    ],
}
# B: sizes that fill whole tiles of the matrix-unit kernels; a window of whole pages; one expert chosen.
BB = {
    "architecture": "Busadra", "vocab": 300, "width": 128, "norm": {"eps": 1e-5}, "canon": {"taps": 4}, "logit_scale": 1.5,
    "layers": [
        {"type": "hgrn2", "mixer": {"heads": 2, "dim": 64, "vdim": 64}, "mlp": _moe(64, 4, 1)},
        {"type": "attention",
         "mixer": {"heads": 8, "kv_heads": 2, "dim": 64, "vdim": 64, "mask": {"size": 64}, "scale": 0.125, "softcap": 8.0,
                   "rot": {"base": 10000.0, "dims": 64, "scaling": {"factor": 8.0, "low": 1.0, "high": 4.0, "original": 512}}},
         "mlp": _moe(96, 8, 3)},
        {"type": "hgrn2", "mixer": {"heads": 3, "dim": 32, "vdim": 128}, "mlp": _moe(32, 4, 2)},
    ],
}
# C: one head; no taps but the token's own (the convolution keeps nothing); a window of one key; every expert chosen; a
# single layer result in the first average; frequencies without scaling.
BC = {
    "architecture": "Busadra", "vocab": 150, "width": 64, "norm": {"eps": 1e-5}, "canon": {"taps": 1}, "logit_scale": 1.0,
    "layers": [
        {"type": "attention",
         "mixer": {"heads": 1, "kv_heads": 1, "dim": 32, "vdim": 48, "mask": {"size": 4096}, "scale": 0.2, "softcap": 2.0,
                   "rot": {"base": 500.0, "dims": 4}},
         "mlp": _moe(32, 3, 3)},
        {"type": "attention",
         "mixer": {"heads": 6, "kv_heads": 1, "dim": 8, "vdim": 8, "mask": {"size": 1}, "scale": 0.3, "softcap": 30.0,
                   "rot": {"base": 100.0, "dims": 8, "scaling": {"factor": 3.0, "low": 2.0, "high": 2.0, "original": 100}}},
         "mlp": _moe(40, 2, 1)},
        {"type": "hgrn2", "mixer": {"heads": 1, "dim": 16, "vdim": 8}, "mlp": _moe(16, 1, 1)},
    ],
}
# D: sizes that fill no tile of any kernel: a width of 70, heads of 6 and 10, six taps, experts of 20 and of 30.
BD = {
    "architecture": "Busadra", "vocab": 97, "width": 70, "norm": {"eps": 1e-4}, "canon": {"taps": 6}, "logit_scale": 3.0,
    "layers": [
        {"type": "hgrn2", "mixer": {"heads": 5, "dim": 6, "vdim": 10}, "mlp": _moe(20, 7, 2)},
        {"type": "hgrn2", "mixer": {"heads": 1, "dim": 3, "vdim": 7}, "mlp": _moe(30, 3, 2)},
        {"type": "attention",
         "mixer": {"heads": 6, "kv_heads": 3, "dim": 10, "vdim": 6, "mask": {"size": 21}, "scale": 0.4, "softcap": 6.0,
                   "rot": {"base": 300.0, "dims": 6, "scaling": {"factor": 1.5, "low": 1.0, "high": 8.0, "original": 40}}},
         "mlp": _moe(20, 3, 1)},
        {"type": "hgrn2", "mixer": {"heads": 2, "dim": 22, "vdim": 5}, "mlp": _moe(20, 2, 2)},
    ],
}
TINY = {"A": (BA, 21, 8), "B": (BB, 22, 16), "C": (BC, 23, 4), "D": (BD, 24, 2)}      # config, seed, page size


def random_config(seed):
    """A Busadra configuration drawn at random: two to seven layers of the two mixers in any order, head counts, sizes,
    windows, constants and mixtures drawn independently."""
    rng = random.Random(seed)
    width = rng.choice([64, 80, 96, 128, 160, 192, 250, 256, 384, 512])
    layers = []
    for _ in range(rng.randint(2, 7)):
        heads = rng.choice([1, 2, 3, 5, 8, 10, 12, 16])
        vdim = rng.choice([8, 16, 24, 40, 48, 64, 96, 128, 160])
        if rng.random() < 0.6:
            layer = {"type": "hgrn2", "mixer": {"heads": heads, "dim": rng.choice([8, 14, 16, 24, 32, 56, 64, 96, 128, 160, 200]),
                                                "vdim": vdim}}
        else:
            dim = rng.choice([8, 16, 24, 32, 40, 64, 80, 96, 128])
            kvh = rng.choice([d for d in (1, 2, 3, 4, 5, 8, 12, 16) if heads % d == 0])
            rot = {"base": rng.choice([100.0, 10000.0, 50000.0, 1e6]), "dims": rng.choice([d for d in (2, 4, 8, 16, 32, 64, 128) if d <= dim]),
                   "scaling": {"factor": rng.choice([1.0, 2.0, 8.0, 32.0]), "low": rng.choice([0.5, 1.0, 2.0]),
                               "high": rng.choice([2.5, 4.0, 16.0]), "original": rng.choice([32, 256, 2048, 8192])}}
            layer = {"type": "attention",
                     "mixer": {"heads": heads, "kv_heads": kvh, "dim": dim, "vdim": min(vdim, 128), "scale": 1.5 * dim ** -0.5,
                               "softcap": rng.choice([1.0, 5.0, 30.0, 50.0]), "mask": {"size": rng.randint(1, 300)}, "rot": rot}}
        e = rng.choice([1, 2, 3, 5, 16, 24, 64, 96])
        layer["mlp"] = _moe(rng.choice([16, 24, 32, 64, 100, 128, 160]), e, rng.randint(1, min(e, 8))) if rng.random() < 0.92 else None
        layers.append(layer)
    return {"architecture": "Busadra", "vocab": rng.choice([128, 300, 512, 1000]), "width": width,
            "norm": {"eps": rng.choice([1e-6, 1e-5, 1e-3])}, "canon": {"taps": rng.choice([1, 2, 3, 4, 5, 7])},
            "logit_scale": rng.choice([0.25, 1.0, 4.0]), "layers": layers}


def tensor_shapes(cfg):
    """name -> (shape, kind of values) of every tensor of a configuration, from the design's naming."""
    w, taps = cfg["width"], cfg["canon"]["taps"]
    out = {"embed": ((cfg["vocab"], w), "embed"), "final.norm": ((w,), "gains"), "head": ((cfg["vocab"], w), "matrix")}
    for i, layer in enumerate(cfg["layers"]):
        m, p, mlp = layer["mixer"], f"l{i}", layer["mlp"]
        h, d, dv = m["heads"], m["dim"], m["vdim"]
        out[f"{p}.norm1"] = ((w,), "gains")
        out[f"{p}.canon1"] = ((w, taps), "taps")
        out[f"{p}.ls1"] = ((w,), "scale")
        out[f"{p}.dwa"] = ((i + 2,), "average")
        if layer["type"] == "hgrn2":
            out[f"{p}.mix.q"] = ((h * d, w), "matrix")
            out[f"{p}.mix.f"] = ((h * d, w), "matrix")
            out[f"{p}.mix.f.b"] = ((h * d,), "gate")
            out[f"{p}.mix.lower"] = ((h * d,), "lower")
            out[f"{p}.mix.v"] = ((h * dv, w), "matrix")
            out[f"{p}.mix.norm"] = ((dv,), "gains")
        else:
            for n, rows in (("q", h * d), ("k", m["kv_heads"] * d), ("v", m["kv_heads"] * dv)):
                out[f"{p}.mix.{n}"] = ((rows, w), "matrix")
                out[f"{p}.mix.{n}.b"] = ((rows,), "bias")
            out[f"{p}.mix.o.b"] = ((w,), "bias")
        out[f"{p}.mix.o"] = ((w, h * dv), "matrix")
        if mlp is None:
            continue
        out[f"{p}.norm2"] = ((w,), "gains")
        out[f"{p}.canon2"] = ((w, taps), "taps")
        out[f"{p}.ls2"] = ((w,), "scale")
        f = mlp["expert"]["ff"]
        out[f"{p}.mlp.router"] = ((mlp["router"]["experts"], w), "router")
        for e in range(mlp["router"]["experts"]):
            out[f"{p}.mlp.e{e}.gate"] = ((f, w), "matrix")
            out[f"{p}.mlp.e{e}.up"] = ((f, w), "matrix")
            out[f"{p}.mlp.e{e}.down"] = ((w, f), "matrix")
    return out


def random_tensors(cfg, seed, dtype=torch.bfloat16):
    g = torch.Generator().manual_seed(seed)
    out = {}
    for name, (shape, kind) in tensor_shapes(cfg).items():
        n = lambda *s: torch.randn(*s, generator=g)
        if kind == "embed":
            t = n(*shape)
        elif kind == "matrix":
            t = n(*shape) * (1.3 / math.sqrt(shape[-1]))
        elif kind == "router":
            t = n(*shape) * (2.5 / math.sqrt(shape[-1]))
        elif kind == "bias":
            t = 0.4 * n(*shape)
        elif kind == "gate":
            t = 2.0 + 2.0 * n(*shape)
        elif kind == "lower":
            t = 0.95 * torch.rand(*shape, generator=g)
        elif kind == "taps":
            t = 0.4 * n(*shape)
        elif kind == "scale":
            t = 0.6 + 0.3 * n(*shape)
        elif kind == "average":
            t = 0.35 * n(*shape)
            t[-1] += 0.8
        elif kind == "gains":
            t = 1.0 + 0.3 * n(*shape)
        out[name] = t.to(dtype)
    return out


def write_folder(folder, cfg, tensors):
    from safetensors.torch import save_file
    os.makedirs(folder, exist_ok=True)
    with open(os.path.join(folder, "config.json"), "w") as f:
        json.dump(cfg, f)
    save_file({k: v.contiguous() for k, v in tensors.items()}, os.path.join(folder, "model.safetensors"))
    return folder


def make_folder(tmp, which, dtype=torch.bfloat16):
    cfg, seed, _ = TINY[which]
    return write_folder(os.path.join(str(tmp), f"busadra_{which}"), cfg, random_tensors(cfg, seed, dtype))
