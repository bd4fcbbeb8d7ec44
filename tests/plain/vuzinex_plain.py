"""The Vuzinex decoder, plainly: whole sequences, one function a mechanism, 64-bit by default, nothing shared with
the engine.  An embedding to which a second table's row for the pair (previous token, token) is added; layers with a norm
before and after every sublayer and one factor on what a sublayer gives; some of the layers run several times in a row.
Three mixers: grouped attention in chunks with a sink beside an mLSTM, normed and gated grouped attention beside
gated linear attention, and Mamba-2.  The feed-forward is gated, with biases.  The head is the embedding table.

Notation: T tokens, W width, H heads, G key/value heads, d query/key numbers a head, dv values a head.
"""
from __future__ import annotations

import json
import math
import os
from typing import Dict, List, Optional, Tuple

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


# ---- small things --------------------------------------------------------------------------------------------
def unit(x: torch.Tensor, eps: float) -> torch.Tensor:
    """x / sqrt(mean(x^2) + eps) over the last dimension."""
    return x / torch.sqrt((x * x).sum(dim=-1, keepdim=True) / x.shape[-1] + eps)


def norm_around_one(x: torch.Tensor, w: torch.Tensor, eps: float) -> torch.Tensor:
    return unit(x, eps) * (1.0 + w)


def sigmoid(z: torch.Tensor) -> torch.Tensor:
    return torch.exp(log_sigmoid(z))


def log_sigmoid(z: torch.Tensor) -> torch.Tensor:
    return torch.clamp(z, max=0.0) - torch.log1p(torch.exp(-z.abs()))


def softplus(z: torch.Tensor) -> torch.Tensor:
    return -log_sigmoid(-z)


def silu(z: torch.Tensor) -> torch.Tensor:
    return z * sigmoid(z)


# ---- embedding -----------------------------------------------------------------------------------------------
def bigram_rows(tokens: List[int], buckets: int, mul_prev: int, mul_cur: int) -> List[int]:
    """The row of the second table for every token: the last one (number ``buckets``) for the first token."""
    return [buckets] + [(a * mul_prev + b * mul_cur) % buckets for a, b in zip(tokens, tokens[1:])]


def embed(cfg: dict, w: Dict[str, torch.Tensor], tokens: List[int], dtype) -> torch.Tensor:
    e, b = cfg["embedding"], cfg["embedding"]["bigram"]
    x = w["embed"].to(dtype)[torch.tensor(tokens)] * float(e["scale"])
    return x + w["bigram"].to(dtype)[torch.tensor(bigram_rows(tokens, int(b["buckets"]), int(b["mul_prev"]), int(b["mul_cur"])))]


# ---- positions -----------------------------------------------------------------------------------------------
def banded(base: float, dims: int, sc: Optional[dict]) -> Tuple[List[float], float]:
    """(dims / 2 frequencies, factor on cosine and sine): base^(-2 i / dims), by bands of wavelengths if scaled."""
    out = []
    for i in range(dims // 2):
        f = base ** (-2.0 * i / dims)
        if sc:
            length, orig = 2.0 * math.pi / f, float(sc["original"])
            lo, hi, factor = float(sc["low"]), float(sc["high"]), float(sc["factor"])
            if length > orig / lo:
                f = f / factor
            elif not length < orig / hi:
                s = (orig / length - lo) / (hi - lo)
                f = (1.0 - s) * f / factor + s * f
        out.append(f)
    return out, 1.0


def yarn(base: float, dims: int, sc: Optional[dict]) -> Tuple[List[float], float]:
    """The same under YaRN: a ramp over the index of the frequency between those that turn ``fast`` and ``slow`` times
    in the original length; cosine and sine are multiplied by 0.1 ln(factor) + 1."""
    f = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
    if not sc:
        return f, 1.0
    factor, orig = float(sc["factor"]), float(sc["original"])
    at = lambda turns: dims * math.log(orig / (2.0 * math.pi * turns)) / (2.0 * math.log(base))
    lo, hi = max(math.floor(at(float(sc["fast"]))), 0), min(math.ceil(at(float(sc["slow"]))), dims - 1)
    out = []
    for i, x in enumerate(f):
        r = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(x / factor * r + x * (1.0 - r))
    return out, 0.1 * math.log(factor) + 1.0


def rotate_neighbours(v: torch.Tensor, pos: torch.Tensor, freq: List[float], gain: float) -> torch.Tensor:
    """v [T, heads, n]: numbers 2 i and 2 i + 1 are a pair, turned by pos * freq[i]; numbers beyond the pairs pass."""
    n = 2 * len(freq)
    a = pos.to(torch.float64)[:, None, None] * torch.tensor(freq, dtype=torch.float64)[None, None, :]
    c, s = (torch.cos(a) * gain).to(v.dtype), (torch.sin(a) * gain).to(v.dtype)
    x, y = v[..., 0:n:2], v[..., 1:n:2]
    out = v.clone()
    out[..., 0:n:2] = x * c - y * s
    out[..., 1:n:2] = y * c + x * s
    return out


# ---- attention -----------------------------------------------------------------------------------------------
def softmax_seen(s: torch.Tensor, seen: torch.Tensor, sink: Optional[torch.Tensor] = None) -> torch.Tensor:
    """exp(s) over the seen entries divided by their sum, to which exp(sink) is added if there is one."""
    s = s.masked_fill(~seen, -math.inf)
    m = s.max(dim=-1, keepdim=True).values
    if sink is not None:
        m = torch.maximum(m, sink)
    e = torch.exp(s - m)
    total = e.sum(dim=-1, keepdim=True)
    if sink is not None:
        total = total + torch.exp(sink - m)
    return e / total


def attend(q, k, v, scale: float, seen: torch.Tensor, sink: Optional[torch.Tensor] = None) -> torch.Tensor:
    """q [T, H, d], k [T, G, d], v [T, G, dv] -> [T, H * dv]; sink [H] or None."""
    T, H = q.shape[:2]
    G = k.shape[1]
    out = torch.zeros(T, H, v.shape[2], dtype=q.dtype)
    for h in range(H):
        g = h // (H // G)
        p = softmax_seen((q[:, h] @ k[:, g].T) * scale, seen, None if sink is None else sink[h])
        out[:, h] = p @ v[:, g]
    return out.reshape(T, -1)


def chunk_mask(T: int, size: Optional[int]) -> torch.Tensor:
    i, j = torch.arange(T)[:, None], torch.arange(T)[None, :]
    seen = j <= i
    return seen & (i // size == j // size) if size else seen


def attention_in_chunks(h, pos, w, pre: str, m: dict, eps: float) -> torch.Tensor:
    T = h.shape[0]
    H, G, d, dv = int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"])
    t = lambda n: w[pre + n].to(h.dtype)
    q, k, v = (h @ t("q").T).view(T, H, d), (h @ t("k").T).view(T, G, d), (h @ t("v").T).view(T, G, dv)
    rot = m.get("rot")
    if rot:
        freq, gain = banded(float(rot["base"]), int(rot["dims"]), rot.get("scaling"))
        q, k = rotate_neighbours(q, pos, freq, gain), rotate_neighbours(k, pos, freq, gain)
    size = int(m["mask"]["size"]) if m.get("mask") else None
    return attend(q, k, v, float(m["scale"]), chunk_mask(T, size), t("sink")) @ t("o").T


def attention_normed(h, pos, w, pre: str, m: dict, eps: float) -> torch.Tensor:
    T = h.shape[0]
    H, G, d, dv = int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"])
    t = lambda n: w[pre + n].to(h.dtype)
    q = (h @ t("q").T + t("q.b")).view(T, H, d)
    k = (h @ t("k").T + t("k.b")).view(T, G, d)
    v = (h @ t("v").T + t("v.b")).view(T, G, dv)
    q, k = unit(q, eps) * t("q.norm"), unit(k, eps) * t("k.norm")
    rot = m.get("rot")
    if rot:
        freq, gain = yarn(float(rot["base"]), int(rot["dims"]), rot.get("scaling"))
        q, k = rotate_neighbours(q, pos, freq, gain), rotate_neighbours(k, pos, freq, gain)
    a = attend(q, k, v, float(m["scale"]), chunk_mask(T, None))
    return (a * sigmoid(h @ t("g").T)) @ t("o").T


# ---- recurrences, token by token -----------------------------------------------------------------------------
def matrix_memory(q, k, v, i, f, state=None):
    """q, k [T, H, d], v [T, H, dv], i and f (log gates) [T, H].  Returns (o [T, H, dv], (S, n, m))."""
    T, H, d = q.shape
    dv = v.shape[2]
    if state is None:
        state = (torch.zeros(H, d, dv, dtype=q.dtype), torch.zeros(H, d, dtype=q.dtype), torch.zeros(H, dtype=q.dtype))
    S, n, m = state
    out = torch.zeros(T, H, dv, dtype=q.dtype)
    for t in range(T):
        new = torch.maximum(f[t] + m, i[t])
        keep, write = torch.exp(f[t] + m - new), torch.exp(i[t] - new)
        S = keep[:, None, None] * S + write[:, None, None] * k[t][:, :, None] * v[t][:, None, :]
        n = keep[:, None] * n + write[:, None] * k[t]
        m = new
        den = torch.maximum((n * q[t]).sum(dim=-1).abs(), torch.exp(-m)) + 1e-6
        out[t] = (S * q[t][:, :, None]).sum(dim=1) / den[:, None]
    return out, (S, n, m)


def mlstm(h, w, pre: str, m: dict, eps: float) -> torch.Tensor:
    T = h.shape[0]
    H, d, dv, cap = int(m["heads"]), int(m["dim"]), int(m["vdim"]), float(m["gate_cap"])
    t = lambda n: w[pre + n].to(h.dtype)
    q, k, v = (h @ t("q").T).view(T, H, d) * d ** -0.5, (h @ t("k").T).view(T, H, d), (h @ t("v").T).view(T, H, dv)
    i = cap * torch.tanh((h @ t("i").T + t("i.b")) / cap)
    f = log_sigmoid(cap * torch.tanh((h @ t("f").T + t("f.b")) / cap))
    o, _ = matrix_memory(q, k, v, i, f)
    return (unit(o, eps).reshape(T, H * dv) * t("norm") * sigmoid(h @ t("g").T)) @ t("o").T


def decayed_outer(q, k, v, alpha, S=None):
    """S <- diag(alpha_t) S + k_t v_t^T, o_t = S^T q_t; alpha [T, H, d]."""
    T, H, d = q.shape
    if S is None:
        S = torch.zeros(H, d, v.shape[2], dtype=q.dtype)
    out = torch.zeros(T, H, v.shape[2], dtype=q.dtype)
    for t in range(T):
        S = alpha[t][:, :, None] * S + k[t][:, :, None] * v[t][:, None, :]
        out[t] = (S * q[t][:, :, None]).sum(dim=1)
    return out, S


def gated_linear(h, w, pre: str, m: dict, eps: float) -> torch.Tensor:
    T = h.shape[0]
    H, d, dv, tau = int(m["heads"]), int(m["dim"]), int(m["vdim"]), float(m["tau"])
    t = lambda n: w[pre + n].to(h.dtype)
    q, k, v = (h @ t("q").T).view(T, H, d) * d ** -0.5, (h @ t("k").T).view(T, H, d), (h @ t("v").T).view(T, H, dv)
    z = (h @ t("a1").T) @ t("a2").T + t("a2.b")
    o, _ = decayed_outer(q, k, v, torch.exp(log_sigmoid(z) / tau).view(T, H, d))
    return ((unit(o, eps) * t("norm")).reshape(T, H * dv) * silu(h @ t("g").T)) @ t("o").T


def causal_convolution(x: torch.Tensor, w: torch.Tensor, b: torch.Tensor) -> torch.Tensor:
    """x [T, C], w [C, taps], b [C]: out_t = b + sum_j w[:, j] x_(t - taps + 1 + j), nothing before the start."""
    taps = w.shape[1]
    out = b.expand_as(x).clone()
    for t in range(x.shape[0]):
        for j in range(taps):
            s = t - taps + 1 + j
            if s >= 0:
                out[t] = out[t] + w[:, j] * x[s]
    return out


def state_space(x, B, C, dt, A_log, D, S=None):
    """x [T, H, dv], B and C [T, G, N], dt [T, H] (positive): y [T, H, dv], last S [H, N, dv]."""
    T, H, dv = x.shape
    G, N = B.shape[1:]
    if S is None:
        S = torch.zeros(H, N, dv, dtype=x.dtype)
    grp = torch.arange(H) // (H // G)
    y = torch.zeros_like(x)
    for t in range(T):
        keep = torch.exp(-torch.exp(A_log) * dt[t])
        S = keep[:, None, None] * S + dt[t][:, None, None] * B[t][grp][:, :, None] * x[t][:, None, :]
        y[t] = (S * C[t][grp][:, :, None]).sum(dim=1) + D[:, None] * x[t]
    return y, S


def mamba2(h, w, pre: str, m: dict, eps: float) -> torch.Tensor:
    T = h.shape[0]
    H, dv, N, G, parts = int(m["heads"]), int(m["vdim"]), int(m["state"]), int(m["groups"]), int(m["norm_groups"])
    inner = H * dv
    t = lambda n: w[pre + n].to(h.dtype)
    z, xbc, dt = torch.split(h @ t("in").T, [inner, inner + 2 * G * N, H], dim=-1)
    xbc = silu(causal_convolution(xbc, t("conv"), t("conv.b")))
    x, B, C = torch.split(xbc, [inner, G * N, G * N], dim=-1)
    y, _ = state_space(x.reshape(T, H, dv), B.reshape(T, G, N), C.reshape(T, G, N), softplus(dt + t("dt_bias")), t("A_log"), t("D"))
    y = y.reshape(T, inner) * silu(z)
    return (unit(y.view(T, parts, inner // parts), eps).reshape(T, inner) * t("norm")) @ t("o").T


# ---- feed-forward --------------------------------------------------------------------------------------------
def gated_mlp(h, w, pre: str) -> torch.Tensor:
    t = lambda n: w[pre + n].to(h.dtype)
    return (silu(h @ t("gate").T + t("gate.b")) * (h @ t("up").T + t("up.b"))) @ t("down").T + t("down.b")


# ---- the model -----------------------------------------------------------------------------------------------
def layer_order(n: int, loop: Optional[dict]) -> List[int]:
    """The layers in the order in which they run."""
    if not loop:
        return list(range(n))
    a, b = int(loop["start"]), int(loop["stop"])
    return list(range(a)) + list(range(a, b)) * int(loop["times"]) + list(range(b, n))


def mixer(h, pos, w, pre: str, layer: dict, eps: float) -> torch.Tensor:
    m = layer["mixer"]
    if layer["type"] == "mamba2":
        return mamba2(h, w, pre, m, eps)
    left, right = {"parallel": (attention_in_chunks, mlstm), "parallel_2": (attention_normed, gated_linear)}[layer["type"]]
    return float(m["left_scale"]) * left(h, pos, w, pre + "left.", m["left"], eps) + \
        float(m["right_scale"]) * right(h, w, pre + "right.", m["right"], eps)


def forward(cfg: dict, tensors: Dict[str, torch.Tensor], tokens: List[int], dtype=torch.float64,
            layers_out: Optional[list] = None) -> torch.Tensor:
    """Logits [T, vocab] for a whole sequence; ``layers_out`` collects the stream after every run of a layer."""
    w = tensors
    eps, mult = float(cfg["norm"]["eps"]), float(cfg["residual_mult"])
    pos = torch.arange(len(tokens))
    x = embed(cfg, w, tokens, dtype)
    for i in layer_order(len(cfg["layers"]), cfg.get("loop")):
        layer, pre = cfg["layers"][i], f"l{i}."
        n = lambda name: w[pre + name].to(dtype)
        y = mixer(norm_around_one(x, n("norm1"), eps), pos, w, pre + "mix.", layer, eps)
        x = x + mult * norm_around_one(y, n("norm1b"), eps)
        if layer.get("mlp") is not None:
            y = gated_mlp(norm_around_one(x, n("norm2"), eps), w, pre + "mlp.")
            x = x + mult * norm_around_one(y, n("norm2b"), eps)
        if layers_out is not None:
            layers_out.append(x.clone())
    x = norm_around_one(x, w["final.norm"].to(dtype), eps)
    return x @ w["embed"].to(dtype).T * float(cfg["logit_scale"])


def greedy_generate(cfg: dict, tensors: Dict[str, torch.Tensor], prompt: List[int], n: int) -> List[int]:
    tokens, out = list(prompt), []
    for _ in range(n):
        nxt = int(forward(cfg, tensors, tokens)[-1].argmax())
        out.append(nxt)
        tokens.append(nxt)
    return out
