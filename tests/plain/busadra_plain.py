"""The Busadra decoder, plainly: whole sequences, one function a mechanism, 64-bit by default, nothing shared
with the engine.  A pre-norm decoder with a layer norm (weight, no bias) before each sublayer, a causal convolution
added to what each sublayer reads, a learned scale per channel on what each sublayer gives, and after every layer a
weighted sum over the embedding output and all layers' results so far.  Two mixers: HGRN2 (a recurrence whose forget
gate also decides what is written) and grouped attention under a window with capped scores and a 1 added to the
softmax's denominator.  The feed-forward is a mixture of gated experts that scale their input.

Notation: T tokens, W width, H heads, G key/value heads, d query/key numbers a head, dv values a head.
"""
from __future__ import annotations

import json
import math
import os
from typing import Dict, List, Optional

import torch
from safetensors import safe_open


def read_folder(folder: str):
    with open(os.path.join(folder, "config.json")) as f:
        cfg = json.load(f)
    tensors: Dict[str, torch.Tensor] = {}
    for fn in sorted(os.listdir(folder)):
        if fn.endswith(".safetensors"):
            with safe_open(os.path.join(folder, fn), framework="pt", device="cpu") as f:
                for name in f.keys():
                    tensors[name] = f.get_tensor(name)
    return cfg, tensors


# ---- norms ---------------------------------------------------------------------------------------------------
def layer_norm(x: torch.Tensor, w: torch.Tensor, eps: float) -> torch.Tensor:
    """(x - mean) / sqrt(mean of squared deviations + eps) * w over the last dimension."""
    mu = x.sum(dim=-1, keepdim=True) / x.shape[-1]
    dev = x - mu
    return dev * w / torch.sqrt((dev * dev).sum(dim=-1, keepdim=True) / x.shape[-1] + eps)


def rms_norm(x: torch.Tensor, w: torch.Tensor, eps: float) -> torch.Tensor:
    return x * w / torch.sqrt((x * x).sum(dim=-1, keepdim=True) / x.shape[-1] + eps)


# ---- convolution over time, added to its input ------------------------------------------------------------------
def input_convolution(h: torch.Tensor, w: torch.Tensor) -> torch.Tensor:
    """h [T, W], w [W, taps]: out_t = h_t + sum_j w[:, j] h_(t - taps + 1 + j), nothing before the start."""
    taps = w.shape[1]
    out = h.clone()
    for t in range(h.shape[0]):
        for j in range(taps):
            s = t - taps + 1 + j
            if s >= 0:
                out[t] = out[t] + w[:, j] * h[s]
    return out


# ---- positions -----------------------------------------------------------------------------------------------
def frequencies(base: float, dims: int, scaling: Optional[dict]) -> List[float]:
    """dims / 2 frequencies base^(-2 i / dims); with a scaling, those whose wavelength is above original / low are
    divided by factor, those below original / high kept, the ones between blended linearly in original / wavelength."""
    out = []
    for i in range(dims // 2):
        f = base ** (-2.0 * i / dims)
        if scaling:
            length = 2.0 * math.pi / f
            factor, lo, hi = float(scaling["factor"]), float(scaling["low"]), float(scaling["high"])
            orig = float(scaling["original"])
            if length > orig / lo:
                f = f / factor
            elif not length < orig / hi:
                s = (orig / length - lo) / (hi - lo)
                f = (1.0 - s) * f / factor + s * f
        out.append(f)
    return out


def rotate_half_split(v: torch.Tensor, pos: torch.Tensor, freq: List[float]) -> torch.Tensor:
    """v [T, heads, n]: number i < len(freq) pairs with number i + len(freq), turned by pos * freq[i]; the rest passes."""
    half = len(freq)
    a = pos.to(torch.float64)[:, None, None] * torch.tensor(freq, dtype=torch.float64)[None, None, :]
    c, s = torch.cos(a).to(v.dtype), torch.sin(a).to(v.dtype)
    u, w = v[..., :half], v[..., half:2 * half]
    return torch.cat([u * c - w * s, w * c + u * s, v[..., 2 * half:]], dim=-1)


# ---- mixers ------------------------------------------------------------------------------------------------------
def softmax_with_one(s: torch.Tensor) -> torch.Tensor:
    """exp(s) / (1 + sum exp(s)) over the last dimension; -inf entries are not seen."""
    m = torch.clamp(s.max(dim=-1, keepdim=True).values, min=0.0)
    e = torch.exp(s - m)
    return e / (torch.exp(-m) + e.sum(dim=-1, keepdim=True))


def soft_cap(s: torch.Tensor, cap: float) -> torch.Tensor:
    return cap * torch.tanh(s / cap)


def window_attention(h: torch.Tensor, pos: torch.Tensor, w: Dict[str, torch.Tensor], pre: str, m: dict) -> torch.Tensor:
    T = h.shape[0]
    H, G, d, dv = int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"])
    f = lambda n: w[pre + n].to(h.dtype)
    q = (h @ f("q").T + f("q.b")).view(T, H, d)
    k = (h @ f("k").T + f("k.b")).view(T, G, d)
    v = (h @ f("v").T + f("v.b")).view(T, G, dv)
    rot = m["rot"]
    freq = frequencies(float(rot["base"]), int(rot["dims"]), rot.get("scaling"))
    q, k = rotate_half_split(q, pos, freq), rotate_half_split(k, pos, freq)
    i, j = torch.arange(T)[:, None], torch.arange(T)[None, :]
    seen = (j <= i) & (i - j < int(m["mask"]["size"]))
    out = torch.zeros(T, H, dv, dtype=h.dtype)
    for hh in range(H):
        g = hh // (H // G)
        s = soft_cap((q[:, hh] @ k[:, g].T) * float(m["scale"]), float(m["softcap"]))
        out[:, hh] = softmax_with_one(s.masked_fill(~seen, -math.inf)) @ v[:, g]
    return out.reshape(T, H * dv) @ f("o").T + f("o.b")


def hgrn2(h: torch.Tensor, w: Dict[str, torch.Tensor], pre: str, m: dict, eps: float,
          state: Optional[torch.Tensor] = None):
    """Token by token: f = l + (1 - l) sigmoid(W_f h + b), S <- diag(f) S + (1 - f) v^T, o = S^T q; a norm per head,
    the output projection.  Returns (output, last state [H, d, dv])."""
    T = h.shape[0]
    H, d, dv = int(m["heads"]), int(m["dim"]), int(m["vdim"])
    t = lambda n: w[pre + n].to(h.dtype)
    q = h @ t("q").T
    q = (q * torch.sigmoid(q)).view(T, H, d)
    v = (h @ t("v").T).view(T, H, dv)
    low = t("lower")
    z = h @ t("f").T + t("f.b")
    f = (low + (1 - low) * torch.sigmoid(z)).view(T, H, d)
    write = ((1 - low) * torch.sigmoid(-z)).view(T, H, d)
    S = torch.zeros(H, d, dv, dtype=h.dtype) if state is None else state.clone()
    o = torch.zeros(T, H, dv, dtype=h.dtype)
    for n in range(T):
        S = f[n][:, :, None] * S + write[n][:, :, None] * v[n][:, None, :]
        o[n] = (S * q[n][:, :, None]).sum(dim=1)
    o = rms_norm(o, t("norm"), eps)
    return o.reshape(T, H * dv) @ t("o").T, S


# ---- feed-forward ------------------------------------------------------------------------------------------------
def route_sigmoid(z: torch.Tensor, top: int):
    """z [T, E] logits -> (ids [T, top], weights [T, top]): the largest sigmoids, as they are."""
    s = torch.sigmoid(z)
    ids = torch.argsort(z, dim=-1, descending=True, stable=True)[:, :top]
    return ids, torch.gather(s, 1, ids)


def expert(h: torch.Tensor, w: Dict[str, torch.Tensor], pre: str) -> torch.Tensor:
    g = h @ w[pre + "gate"].to(h.dtype).T
    u = h @ w[pre + "up"].to(h.dtype).T
    return (g * torch.sigmoid(g) * u) @ w[pre + "down"].to(h.dtype).T


def mixture(h: torch.Tensor, w: Dict[str, torch.Tensor], pre: str, mlp: dict) -> torch.Tensor:
    """sum over the chosen experts of expert(weight * h)."""
    ids, wts = route_sigmoid(h @ w[pre + "router"].to(h.dtype).T, int(mlp["router"]["top"]))
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for c in range(ids.shape[1]):
            out[t] += expert(wts[t, c] * h[t:t + 1], w, f"{pre}e{int(ids[t, c])}.")[0]
    return out


# ---- the model -----------------------------------------------------------------------------------------------------
def depth_average(coef: torch.Tensor, results: List[torch.Tensor]) -> torch.Tensor:
    """sum_j coef[j] results[j]: results[0] the embedding output, results[i + 1] layer i's."""
    assert coef.shape[0] == len(results)
    out = torch.zeros_like(results[0])
    for c, r in zip(coef, results):
        out = out + c * r
    return out


def forward(cfg: dict, tensors: Dict[str, torch.Tensor], tokens: List[int], dtype=torch.float64,
            layers_out: Optional[list] = None) -> torch.Tensor:
    """Logits [T, vocab] for a whole sequence; ``layers_out`` collects the stream after every layer."""
    w = tensors
    eps = float(cfg["norm"]["eps"])
    pos = torch.arange(len(tokens))
    x = w["embed"].to(dtype)[torch.tensor(tokens)]
    results = [x]
    for i, layer in enumerate(cfg["layers"]):
        pre = f"l{i}."
        f = lambda n: w[pre + n].to(dtype)
        h = input_convolution(layer_norm(x, f("norm1"), eps), f("canon1"))
        if layer["type"] == "hgrn2":
            y, _ = hgrn2(h, w, pre + "mix.", layer["mixer"], eps)
        elif layer["type"] == "attention":
            y = window_attention(h, pos, w, pre + "mix.", layer["mixer"])
        else:
            raise ValueError(layer["type"])
        x = x + f("ls1") * y
        if layer.get("mlp") is not None:
            h = input_convolution(layer_norm(x, f("norm2"), eps), f("canon2"))
            x = x + f("ls2") * mixture(h, w, pre + "mlp.", layer["mlp"])
        results.append(x)
        x = depth_average(f("dwa"), results)
        if layers_out is not None:
            layers_out.append(x.clone())
    x = layer_norm(x, w["final.norm"].to(dtype), eps)
    return x @ w["head"].to(dtype).T * float(cfg["logit_scale"])


def greedy_generate(cfg: dict, tensors: Dict[str, torch.Tensor], prompt: List[int], n: int) -> List[int]:
    tokens, out = list(prompt), []
    for _ in range(n):
        nxt = int(forward(cfg, tensors, tokens)[-1].argmax())
        out.append(nxt)
        tokens.append(nxt)
    return out
