"""Typed configuration of the Vuzinex decoder, read from config.json.

A decoder with norms on both sides of every sublayer: x <- x + r * n1b(mixer(n1(x))), x <- x + r * n2b(ff(n2(x))), RMS
norms whose weights are stored around zero.  The stream begins as a scaled row of the embedding table plus a row of a
second table that the token and the one before it choose; the head is the embedding table, with a factor on the logits.
Some neighbouring layers run several times in a row, every run with a cache and state of its own.  A layer's mixer is one of
  parallel    attention inside chunks of positions, a learned sink per head and rotated neighbouring pairs whose frequencies
              are scaled by bands of wavelengths, beside the matrix memory of xLSTM;
  parallel_2  attention over all keys with biases, q and k normed per head, rotated neighbouring pairs under YaRN and a gate
              on the output, beside gated linear attention;
  mamba2      a state space (Mamba-2).
Two mixers side by side are added with weights.  The feed-forward is gated, with biases, or absent.

Keys: architecture, vocab, width, norm.eps, residual_mult, logit_scale, embedding {scale, bigram {buckets, mul_prev,
mul_cur}}, loop {start, stop, times} (or none), layers[i].type, layers[i].mlp (null | {kind: dense, ff}), layers[i].mixer:
  parallel    {left {heads, kv_heads, dim, vdim, scale, mask {size}, rot {base, dims, scaling {factor, low, high, original}}},
              right {heads, dim, vdim, gate_cap}, left_scale, right_scale}
  parallel_2  {left {heads, kv_heads, dim, vdim, scale, rot {base, dims, scaling {factor, original, fast, slow}}},
              right {heads, dim, vdim, tau} (+ decay_rank, else the rows of the layer's tensor mix.right.a1), left_scale,
              right_scale}
  mamba2      {heads, vdim, state, groups, conv, norm_groups}
No size has a default.  The one size that only a tensor's shape gives is written into the dictionary that ``to_dict`` returns.
"""
from __future__ import annotations

import copy
from typing import Any, Dict, List, Optional, Tuple

from .qwen3 import ConfigError
from .spec import (BareRMSNormSpec, ChunkAttentionSpec, GatedLinearSpec, MatrixMemorySpec, ModelSpec, PairEmbeddingSpec,
                   RopePairsSpec, SandwichLayerSpec, ScheduleEntry, SideBySideMixerSpec, StateSpaceSpec, SwiGLUSpec)

ARCHITECTURE = "Vuzinex"
MIXERS = ("parallel", "parallel_2", "mamba2")
MAX_POSITIONS = 1 << 20      # the design names no limit; positions stay exact in 32-bit floats far beyond this
MAX_KEY_CHANNELS = 256       # what the kernels of the recurrences take


def _get(d: Dict[str, Any], path: str, where: str):
    cur: Any = d
    for key in path.split("."):
        if not isinstance(cur, dict) or key not in cur:
            raise ConfigError(f"config.json lacks {where}{path}")
        cur = cur[key]
    return cur


def _sizes(m: Dict[str, Any], where: str, *names: str) -> List[int]:
    out = []
    for name in names:
        v = int(_get(m, name, where))
        if v <= 0:
            raise ConfigError(f"{where}{name} = {v} must be positive")
        out.append(v)
    return out


class VuzinexConfig:
    architecture = ARCHITECTURE

    def __init__(self, d: Dict[str, Any], shapes: Optional[Dict[str, Tuple[int, ...]]] = None):
        self.raw = copy.deepcopy(d)
        self.vocab, self.width = _sizes(d, "", "vocab", "width")
        self.eps = float(_get(d, "norm.eps", ""))
        self.residual_mult = float(_get(d, "residual_mult", ""))
        self.logit_scale = float(_get(d, "logit_scale", ""))
        self.embedding_scale = float(_get(d, "embedding.scale", ""))
        self.buckets, = _sizes(_get(d, "embedding.bigram", ""), "embedding.bigram.", "buckets")
        self.mul_prev, self.mul_cur = (int(_get(d, "embedding.bigram." + k, "")) for k in ("mul_prev", "mul_cur"))
        _get(d, "layers", "")
        self.layers: List[Dict[str, Any]] = self.raw["layers"]      # (the size found in a tensor's shape is written here)
        self.loop = d.get("loop")
        self.max_positions = int(d.get("max_positions", MAX_POSITIONS))
        for i, layer in enumerate(self.layers):
            right = layer["mixer"].get("right") if layer.get("type") == "parallel_2" and isinstance(layer.get("mixer"), dict) else None
            name = f"l{i}.mix.right.a1"
            if isinstance(right, dict) and "decay_rank" not in right and shapes and name in shapes:
                right["decay_rank"] = int(shapes[name][0])
        self.validate()

    @classmethod
    def from_dict(cls, d: Dict[str, Any], shapes: Optional[Dict[str, Tuple[int, ...]]] = None) -> "VuzinexConfig":
        return cls(d, shapes)

    def to_dict(self) -> Dict[str, Any]:
        return copy.deepcopy(self.raw)

    def validate(self) -> None:
        if not self.eps > 0:
            raise ConfigError("norm.eps must be positive")
        if not self.layers:
            raise ConfigError("the model has no layers")
        for i, layer in enumerate(self.layers):
            where = f"layers[{i}]."
            if layer.get("type") not in MIXERS:
                raise ConfigError(f"{where}type is {layer.get('type')!r}; known: {', '.join(MIXERS)}")
            self._mixer(layer, where)
            self._ffn(layer, where)
        self.layer_order()

    def layer_order(self) -> List[int]:
        """The layers in the order in which they run."""
        n = len(self.layers)
        if self.loop is None:
            return list(range(n))
        start, stop, times = (int(_get(self.loop, k, "loop.")) for k in ("start", "stop", "times"))
        if not 0 <= start <= stop <= n or times < 1:
            raise ConfigError(f"loop: layers {start} to {stop} of {n}, {times} times")
        return list(range(start)) + list(range(start, stop)) * times + list(range(stop, n))

    # ---- one layer's parts ---------------------------------------------------------------------------------
    @staticmethod
    def _rot(m: Dict[str, Any], where: str, dim: int, keys: Tuple[str, ...], kind: str) -> Optional[RopePairsSpec]:
        rot = m.get("rot")
        dims = int(_get(rot, "dims", where + "rot.")) if rot is not None else 0
        if dims == 0:
            return None
        if dims % 2 or not 0 < dims <= dim:
            raise ConfigError(f"{where}rot.dims = {dims} must be even and at most dim = {dim}")
        scaling = None
        if rot.get("scaling") is not None:
            scaling = tuple(float(_get(rot["scaling"], k, where + "rot.scaling.")) for k in keys)
            if not all(v > 0 for v in scaling):
                raise ConfigError(f"{where}rot.scaling: all of {', '.join(keys)} must be positive")
        return RopePairsSpec(theta=float(_get(rot, "base", where + "rot.")), rotary_dim=dims, **{kind: scaling})

    def _left(self, m: Dict[str, Any], where: str, second: bool) -> ChunkAttentionSpec:
        heads, kv_heads, dim, vdim = _sizes(m, where, "heads", "kv_heads", "dim", "vdim")
        if heads % kv_heads:
            raise ConfigError(f"{where}{heads} heads over {kv_heads} key/value heads")
        sizes = dict(num_heads=heads, num_kv_heads=kv_heads, head_dim=dim, v_head_dim=vdim, scale=float(_get(m, "scale", where)))
        if second:
            return ChunkAttentionSpec(**sizes, bias=True, out_bias=False, qk_norm="head", qk_norm_eps=self.eps, output_gate=True,
                                      position=self._rot(m, where, dim, ("factor", "original", "fast", "slow"), "yarn"))
        mask = m.get("mask")
        return ChunkAttentionSpec(**sizes, chunk=_sizes(mask, where + "mask.", "size")[0] if mask is not None else None, head_sink=True,
                                  position=self._rot(m, where, dim, ("factor", "low", "high", "original"), "band_scaling"))

    def _mixer(self, layer: Dict[str, Any], where: str):
        m, w = _get(layer, "mixer", where), where + "mixer."
        if layer["type"] == "mamba2":
            heads, vdim, state, groups, taps, parts = _sizes(m, w, "heads", "vdim", "state", "groups", "conv", "norm_groups")
            if heads % groups:
                raise ConfigError(f"{w}{heads} heads in {groups} groups")
            if (heads * vdim) % parts:
                raise ConfigError(f"{w}{heads * vdim} numbers in norm_groups = {parts} parts")
            self._channels(state, w + "state")
            return StateSpaceSpec(num_heads=heads, head_dim=vdim, state_dim=state, groups=groups, taps=taps, norm_groups=parts,
                                  norm_eps=self.eps)
        second = layer["type"] == "parallel_2"
        right, wr = _get(m, "right", w), w + "right."
        heads, dim, vdim = _sizes(right, wr, "heads", "dim", "vdim")
        self._channels(dim, wr + "dim")
        sizes = dict(num_heads=heads, head_dim=dim, v_head_dim=vdim, norm_eps=self.eps)
        if second:
            if right.get("decay_rank") is None:
                raise ConfigError(f"config.json lacks {wr}decay_rank, and no tensor's shape was at hand to give it")
            tau = float(_get(right, "tau", wr))
            if not tau > 0:
                raise ConfigError(f"{wr}tau must be positive")
            right_spec = GatedLinearSpec(**sizes, decay_rank=_sizes(right, wr, "decay_rank")[0], tau=tau)
        else:
            cap = float(_get(right, "gate_cap", wr))
            if not cap > 0:
                raise ConfigError(f"{wr}gate_cap must be positive")
            right_spec = MatrixMemorySpec(**sizes, gate_cap=cap)
        return SideBySideMixerSpec(left=self._left(_get(m, "left", w), w + "left.", second), right=right_spec,
                                   left_scale=float(_get(m, "left_scale", w)), right_scale=float(_get(m, "right_scale", w)))

    @staticmethod
    def _channels(n: int, what: str) -> None:
        if n > MAX_KEY_CHANNELS:
            raise ConfigError(f"{what} = {n}: at most {MAX_KEY_CHANNELS}")

    @staticmethod
    def _ffn(layer: Dict[str, Any], where: str) -> Optional[SwiGLUSpec]:
        mlp = layer.get("mlp")
        if mlp is None:
            return None
        w = where + "mlp."
        if _get(mlp, "kind", w) != "dense":
            raise ConfigError(f"{w}kind is {mlp['kind']!r}; known: dense")
        return SwiGLUSpec(intermediate_size=_sizes(mlp, w, "ff")[0], names=("gate", "up", "down"), bias=True)

    # ---- the model this configuration describes --------------------------------------------------------------
    def to_model_spec(self) -> ModelSpec:
        norm = BareRMSNormSpec(eps=self.eps, offset=1.0)
        layers = []
        for i, layer in enumerate(self.layers):
            where = f"layers[{i}]."
            layers.append(SandwichLayerSpec(prefix=f"l{i}", mixer_norm=norm, mixer=self._mixer(layer, where), mixer_post=norm,
                                            ffn_norm=norm, ffn=self._ffn(layer, where), ffn_post=norm, mult=self.residual_mult))
        spec = ModelSpec(
            architecture=self.architecture, vocab_size=self.vocab, hidden_size=self.width, layers=tuple(layers),
            schedule=tuple(ScheduleEntry(layer=i) for i in self.layer_order()),
            final_norm=BareRMSNormSpec(eps=self.eps, offset=1.0, gain=self.logit_scale), embed_name="embed",
            final_norm_name="final.norm", head_name="embed", tie_head=True, max_positions=self.max_positions,
            stream_prologue=PairEmbeddingSpec(scale=self.embedding_scale, buckets=self.buckets, mul_prev=self.mul_prev,
                                              mul_cur=self.mul_cur))
        spec.validate()
        return spec
