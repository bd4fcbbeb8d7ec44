"""Tiny Vuzinex configurations for tests, with random weights of a scale at which every mechanism moves the logits (scores
large enough to prefer keys, sinks that take a good part of the softmax, gates and decays from near 0 to near 1, input
gates on both sides of the running maximum's start), written as model folders.  Sizes differ from one another wherever
the design allows."""
import json
import math
import os
import random

import torch


def _mlp(ff):
    return {"kind": "dense", "ff": ff}


def _one(left, right, ls, rs, mlp):
    return {"type": "parallel", "mixer": {"left": left, "right": right, "left_scale": ls, "right_scale": rs}, "mlp": mlp}


def _two(left, right, ls, rs, mlp):
    return dict(_one(left, right, ls, rs, mlp), type="parallel_2")


def _ssm(heads, vdim, state, groups, conv, parts, mlp=None):
    return {"type": "mamba2", "mixer": {"heads": heads, "vdim": vdim, "state": state, "groups": groups, "conv": conv,
                                        "norm_groups": parts}, "mlp": mlp}


def _cfg(vocab, width, eps, mult, logit, scale, buckets, muls, loop, layers):
    return {"architecture": "Vuzinex", "vocab": vocab, "width": width, "norm": {"eps": eps}, "residual_mult": mult, "logit_scale": logit,
            "embedding": {"scale": scale, "bigram": {"buckets": buckets, "mul_prev": muls[0], "mul_cur": muls[1]}}, "loop": loop,
            "layers": layers}


# A: all three mixers, key and value sizes that differ, grouped heads, rotations of a part of a head, two groups in the
# state space and three norm groups, one of its layers with a feed-forward; layers 1 and 2 run twice.
VA = _cfg(211, 96, 1e-6, 0.6, 0.7, 1.5, 101, (7, 13), {"start": 1, "stop": 3, "times": 2}, [
    _one({"heads": 6, "kv_heads": 2, "dim": 20, "vdim": 12, "scale": 0.4, "mask": {"size": 37},
          "rot": {"base": 500.0, "dims": 12, "scaling": {"factor": 6.0, "low": 1.0, "high": 4.0, "original": 64}}},
         {"heads": 3, "dim": 12, "vdim": 20, "gate_cap": 9.0}, 1.3, 0.4, _mlp(40)),
    _ssm(6, 10, 14, 2, 3, 3),
    _two({"heads": 4, "kv_heads": 4, "dim": 16, "vdim": 24, "scale": 0.5,
          "rot": {"base": 1000.0, "dims": 12, "scaling": {"factor": 3.0, "original": 90, "fast": 8.0, "slow": 1.0}}},
         {"heads": 2, "dim": 28, "vdim": 16, "tau": 5.0, "decay_rank": 9}, 0.8, 1.7, None),
    _ssm(4, 16, 20, 1, 4, 1, _mlp(56)),
])
# B: sizes that fill whole tiles of the matrix-unit kernels; a chunk of whole pages; the first two layers run three times.
VB = _cfg(300, 128, 1e-5, 0.8, 1.0, 2.0, 251, (37, 11), {"start": 0, "stop": 2, "times": 3}, [
    _two({"heads": 8, "kv_heads": 2, "dim": 64, "vdim": 64, "scale": 0.2,
          "rot": {"base": 10000.0, "dims": 64, "scaling": {"factor": 2.0, "original": 128, "fast": 16.0, "slow": 1.0}}},
         {"heads": 2, "dim": 64, "vdim": 64, "tau": 16.0, "decay_rank": 16}, 1.0, 0.5, _mlp(96)),
    _ssm(4, 64, 32, 1, 4, 1),
    _one({"heads": 4, "kv_heads": 2, "dim": 128, "vdim": 128, "scale": 0.15, "mask": {"size": 64},
          "rot": {"base": 1e6, "dims": 128, "scaling": {"factor": 8.0, "low": 1.0, "high": 4.0, "original": 256}}},
         {"heads": 3, "dim": 32, "vdim": 96, "gate_cap": 12.0}, 1.0, 1.0, _mlp(64)),
])
# C: one head; no taps but the token's own (the convolution keeps nothing); a chunk of one key and one beyond every prompt;
# no feed-forward beside attention; no rotation, no scaling of frequencies; as many groups as heads; nothing runs twice.
VC = _cfg(150, 64, 1e-5, 1.0, 2.0, 1.0, 1, (3, 5), None, [
    _one({"heads": 1, "kv_heads": 1, "dim": 32, "vdim": 48, "scale": 0.3, "mask": {"size": 1}},
         {"heads": 1, "dim": 16, "vdim": 8, "gate_cap": 3.0}, 0.5, -0.7, None),
    _two({"heads": 6, "kv_heads": 1, "dim": 8, "vdim": 8, "scale": 0.6, "rot": {"base": 100.0, "dims": 8}},
         {"heads": 1, "dim": 8, "vdim": 16, "tau": 1.0, "decay_rank": 1}, -1.2, 0.6, _mlp(32)),
    _ssm(3, 8, 8, 3, 1, 1),
    _one({"heads": 2, "kv_heads": 1, "dim": 16, "vdim": 16, "scale": 0.5, "mask": {"size": 4096}, "rot": {"base": 500.0, "dims": 4}},
         {"heads": 2, "dim": 8, "vdim": 8, "gate_cap": 20.0}, 1.0, 1.0, _mlp(16)),
])
# D: sizes that fill no tile of any kernel: a width of 70, heads of 6 and 10, three key channels, six taps; all layers run
# twice.
VD = _cfg(97, 70, 1e-4, 0.5, 3.0, 0.7, 53, (1, 1), {"start": 0, "stop": 4, "times": 2}, [
    _ssm(5, 6, 7, 1, 6, 2),
    _one({"heads": 6, "kv_heads": 3, "dim": 10, "vdim": 6, "scale": 0.5, "mask": {"size": 21},
          "rot": {"base": 300.0, "dims": 6, "scaling": {"factor": 1.5, "low": 1.0, "high": 8.0, "original": 40}}},
         {"heads": 2, "dim": 3, "vdim": 7, "gate_cap": 6.0}, 2.0, 0.3, _mlp(20)),
    _two({"heads": 5, "kv_heads": 5, "dim": 6, "vdim": 10, "scale": 0.7,
          "rot": {"base": 50.0, "dims": 2, "scaling": {"factor": 4.0, "original": 30, "fast": 4.0, "slow": 1.0}}},
         {"heads": 3, "dim": 22, "vdim": 5, "tau": 2.5, "decay_rank": 5}, 0.3, 0.9, _mlp(30)),
    _ssm(2, 15, 9, 2, 2, 5, _mlp(24)),
])
TINY = {"A": (VA, 21, 8), "B": (VB, 22, 16), "C": (VC, 23, 4), "D": (VD, 24, 2)}      # config, seed, page size


def random_config(seed):
    """A Vuzinex configuration drawn at random: two to six layers of the three mixers in any order, head counts, sizes,
    chunks and constants drawn independently, and a loop over some of the layers or none."""
    rng = random.Random(seed)
    width = rng.choice([64, 80, 96, 128, 160, 192, 250, 256, 384])
    layers = []
    for _ in range(rng.randint(2, 6)):
        mlp = _mlp(rng.choice([16, 32, 64, 100, 128, 160, 192])) if rng.random() < 0.7 else None
        heads = rng.choice([1, 2, 3, 5, 6, 8, 12])
        kind = rng.choice(["parallel", "parallel_2", "mamba2"])
        if kind == "mamba2":
            vdim = rng.choice([8, 16, 24, 40, 48, 64, 96])
            layers.append(_ssm(heads, vdim, rng.choice([8, 14, 16, 32, 48, 64, 128, 144]), rng.choice([d for d in (1, 2, 3, 4, 6) if heads % d == 0]),
                               rng.choice([1, 2, 3, 4, 5]), rng.choice([d for d in (1, 2, 3, 4, 6, 8) if heads * vdim % d == 0]), mlp))
            continue
        dim, vdim = rng.choice([8, 16, 24, 40, 64, 80, 96, 128]), rng.choice([8, 16, 24, 40, 64, 96, 128])
        left = {"heads": heads, "kv_heads": rng.choice([d for d in (1, 2, 3, 4, 6, 8, 12) if heads % d == 0]), "dim": dim, "vdim": vdim,
                "scale": 1.5 * dim ** -0.5}
        rot = {"base": rng.choice([100.0, 10000.0, 50000.0, 1e6]), "dims": rng.choice([d for d in (2, 4, 8, 16, 32, 64, 128) if d <= dim])}
        right = {"heads": rng.choice([1, 2, 3, 4, 7]), "dim": rng.choice([8, 16, 24, 40, 64, 128, 160]),
                 "vdim": rng.choice([8, 16, 32, 40, 64, 96, 128, 144])}
        scales = (rng.choice([0.5, 1.0, 1.2, 2.0]), rng.choice([0.3, 0.5, 1.0, 1.6]))
        if kind == "parallel":
            rot["scaling"] = {"factor": rng.choice([1.0, 2.0, 8.0]), "low": rng.choice([0.5, 1.0]), "high": rng.choice([2.5, 4.0, 16.0]),
                              "original": rng.choice([32, 256, 2048])}
            layers.append(_one(dict(left, mask={"size": rng.randint(1, 200)}, rot=rot), dict(right, gate_cap=rng.choice([4.0, 8.0, 15.0])),
                               *scales, mlp))
        else:
            rot["scaling"] = {"factor": rng.choice([1.5, 2.0, 8.0]), "original": rng.choice([64, 256, 2048]), "fast": rng.choice([8.0, 32.0]),
                              "slow": rng.choice([1.0, 2.0])}
            layers.append(_two(dict(left, rot=rot), dict(right, tau=rng.choice([1.0, 4.0, 16.0]), decay_rank=rng.choice([1, 4, 8, 16, 24])),
                               *scales, mlp))
    n = len(layers)
    loop = None
    if rng.random() < 0.7:
        start = rng.randrange(n)
        loop = {"start": start, "stop": rng.randint(start + 1, n), "times": rng.choice([1, 2, 3])}
    return _cfg(rng.choice([128, 300, 512]), width, rng.choice([1e-6, 1e-5, 1e-3]), rng.choice([0.4, 0.7, 1.0]), rng.choice([0.25, 1.0, 4.0]),
                rng.choice([0.5, 1.0, 3.0]), rng.choice([7, 101, 499]), (rng.choice([1, 5, 29, 1009]), rng.choice([1, 19, 40])), loop, layers)


def tensor_shapes(cfg):
    """name -> (shape, kind of values) of every tensor of a configuration, from the design's naming."""
    w = cfg["width"]
    out = {"embed": ((cfg["vocab"], w), "embed"), "bigram": ((cfg["embedding"]["bigram"]["buckets"] + 1, w), "embed"),
           "final.norm": ((w,), "around zero")}
    for i, layer in enumerate(cfg["layers"]):
        m, p = layer["mixer"], f"l{i}"
        out[f"{p}.norm1"] = out[f"{p}.norm1b"] = ((w,), "around zero")
        if layer["type"] == "mamba2":
            h, inner, gn = m["heads"], m["heads"] * m["vdim"], m["groups"] * m["state"]
            out[f"{p}.mix.in"] = ((2 * inner + 2 * gn + h, w), "matrix")
            out[f"{p}.mix.conv"] = ((inner + 2 * gn, m["conv"]), "taps")
            out[f"{p}.mix.conv.b"] = ((inner + 2 * gn,), "bias")
            out[f"{p}.mix.dt_bias"] = ((h,), "steps")
            out[f"{p}.mix.A_log"] = ((h,), "bias")
            out[f"{p}.mix.D"] = ((h,), "gains")
            out[f"{p}.mix.norm"] = ((inner,), "gains")
            out[f"{p}.mix.o"] = ((w, inner), "matrix")
        else:
            a, r = m["left"], m["right"]
            pl, pr = f"{p}.mix.left", f"{p}.mix.right"
            for n, rows in (("q", a["heads"] * a["dim"]), ("k", a["kv_heads"] * a["dim"]), ("v", a["kv_heads"] * a["vdim"])):
                out[f"{pl}.{n}"] = ((rows, w), "matrix")
                if layer["type"] == "parallel_2":
                    out[f"{pl}.{n}.b"] = ((rows,), "bias")
            out[f"{pl}.o"] = ((w, a["heads"] * a["vdim"]), "matrix")
            h, nk, nv = r["heads"], r["heads"] * r["dim"], r["heads"] * r["vdim"]
            for n, rows in (("q", nk), ("k", nk), ("v", nv), ("g", nv)):
                out[f"{pr}.{n}"] = ((rows, w), "matrix")
            out[f"{pr}.o"] = ((w, nv), "matrix")
            if layer["type"] == "parallel":
                out[f"{pl}.sink"] = ((a["heads"],), "sink")
                out[f"{pr}.norm"] = ((nv,), "gains")
                out[f"{pr}.i"], out[f"{pr}.f"] = ((h, w), "matrix"), ((h, w), "matrix")
                out[f"{pr}.i.b"], out[f"{pr}.f.b"] = ((h,), "sink"), ((h,), "forget")
            else:
                out[f"{pl}.q.norm"] = out[f"{pl}.k.norm"] = ((a["dim"],), "gains")
                out[f"{pl}.g"] = ((a["heads"] * a["vdim"], w), "matrix")
                out[f"{pr}.norm"] = ((r["vdim"],), "gains")
                out[f"{pr}.a1"], out[f"{pr}.a2"] = ((r["decay_rank"], w), "matrix"), ((nk, r["decay_rank"]), "matrix")
                out[f"{pr}.a2.b"] = ((nk,), "forget")
        if layer["mlp"] is None:
            continue
        f = layer["mlp"]["ff"]
        out[f"{p}.norm2"] = out[f"{p}.norm2b"] = ((w,), "around zero")
        for n, shape in (("gate", (f, w)), ("up", (f, w)), ("down", (w, f))):
            out[f"{p}.mlp.{n}"] = (shape, "matrix")
            out[f"{p}.mlp.{n}.b"] = ((shape[0],), "bias")
    return out


def random_tensors(cfg, seed, dtype=torch.bfloat16):
    g = torch.Generator().manual_seed(seed)
    out = {}
    for name, (shape, kind) in tensor_shapes(cfg).items():
        n = torch.randn(*shape, generator=g)
        out[name] = {"embed": n, "matrix": n * (1.3 / math.sqrt(shape[-1])), "bias": 0.4 * n, "taps": 0.5 * n, "steps": n - 1.5,
                     "sink": 2.0 * n, "forget": 2.0 + 2.0 * n, "gains": 1.0 + 0.3 * n, "around zero": 0.3 * n}[kind].to(dtype)
    return out


def write_folder(folder, cfg, tensors):
    """(config.json without the one size that only a tensor's shape gives)"""
    from safetensors.torch import save_file
    os.makedirs(folder, exist_ok=True)
    cfg = json.loads(json.dumps(cfg))
    for layer in cfg["layers"]:
        if layer["type"] == "parallel_2":
            layer["mixer"]["right"].pop("decay_rank", None)
    with open(os.path.join(folder, "config.json"), "w") as f:
        json.dump(cfg, f)
    save_file({k: v.contiguous() for k, v in tensors.items()}, os.path.join(folder, "model.safetensors"))
    return folder


def make_folder(tmp, which, dtype=torch.bfloat16):
    cfg, seed, _ = TINY[which]
    return write_folder(os.path.join(str(tmp), f"vuzinex_{which}"), cfg, random_tensors(cfg, seed, dtype))
