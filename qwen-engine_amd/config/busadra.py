"""Typed configuration of the Busadra decoder, read from config.json.

A pre-norm decoder: x <- x + s1 * mixer(c1(ln(x))), x <- x + s2 * ff(c2(ln(x))), the norms being layer norms with a
weight and no bias, c1 and c2 causal convolutions over time added to their input, s1 and s2 a learned factor per
channel.  What goes on from a layer is a learned weighted sum over the embedding output and all layers' results so far.
Two mixers, chosen per layer by ``type``:

* ``hgrn2``: a recurrence per head whose forget gate, bounded below, also decides what is written.
* ``attention``: grouped attention under a sliding window with biases, rotated positions scaled by bands of wavelengths,
  softly capped scores and a 1 added to the softmax's denominator.

The feed-forward is a mixture of gated experts; the router's sigmoids choose and weigh, and a weight multiplies what its
expert reads.

Keys: architecture, vocab, width, norm.eps, canon.taps, logit_scale, layers[i].type, layers[i].mixer {heads, dim, vdim,
and for attention: kv_heads, scale, softcap, mask {size}, rot {base, dims, scaling {factor, low, high, original}}},
layers[i].mlp (null | {kind: moe, expert {ff}, router {experts, top}}).  No size has a default.
"""
from __future__ import annotations

import copy
from typing import Any, Dict, List, Optional

from .qwen3 import ConfigError
from .spec import (BareLayerNormSpec, ConvAttentionSpec, DepthAverageSpec, ForgetGateLinearSpec, ModelSpec, RopeHalfAnglesSpec,
                   ScaledLayerSpec, ScheduleEntry, ShortConvSpec, SigmoidMoESpec)

ARCHITECTURE = "Busadra"
MIXER_TYPES = ("hgrn2", "attention")
MAX_POSITIONS = 1 << 20      # the design names no limit; positions stay exact in 32-bit floats far beyond this


def _get(d: Dict[str, Any], path: str, where: str):
    cur: Any = d
    for key in path.split("."):
        if not isinstance(cur, dict) or key not in cur:
            raise ConfigError(f"config.json lacks {where}{path}")
        cur = cur[key]
    return cur


class BusadraConfig:
    architecture = ARCHITECTURE

    def __init__(self, d: Dict[str, Any]):
        self.raw = copy.deepcopy(d)
        self.vocab = int(_get(d, "vocab", ""))
        self.width = int(_get(d, "width", ""))
        self.eps = float(_get(d, "norm.eps", ""))
        self.taps = int(_get(d, "canon.taps", ""))
        self.logit_scale = float(_get(d, "logit_scale", ""))
        self.layers: List[Dict[str, Any]] = list(_get(d, "layers", ""))
        self.max_positions = int(d.get("max_positions", MAX_POSITIONS))
        self.validate()

    @classmethod
    def from_dict(cls, d: Dict[str, Any]) -> "BusadraConfig":
        return cls(d)

    def to_dict(self) -> Dict[str, Any]:
        return copy.deepcopy(self.raw)

    def validate(self) -> None:
        if self.vocab <= 0 or self.width <= 0:
            raise ConfigError("vocab and width must be positive")
        if not self.eps > 0:
            raise ConfigError("norm.eps must be positive")
        if self.taps < 1:
            raise ConfigError("canon.taps must be at least 1")
        if not self.layers:
            raise ConfigError("the model has no layers")
        for i, layer in enumerate(self.layers):
            where = f"layers[{i}]."
            if layer.get("type") not in MIXER_TYPES:
                raise ConfigError(f"{where}type is {layer.get('type')!r}; known: {list(MIXER_TYPES)}")
            self._mixer(layer, where)
            self._ffn(layer, where)

    # ---- one layer's parts --------------------------------------------------------------------------------------
    @staticmethod
    def _rot(m: Dict[str, Any], where: str, most: int) -> Optional[RopeHalfAnglesSpec]:
        rot = m.get("rot")
        if rot is None:
            return None
        w = where + "rot."
        dims = int(_get(rot, "dims", w))
        if dims == 0:
            return None
        if dims % 2 or not 0 < dims <= most:
            raise ConfigError(f"{w}dims = {dims} must be even and at most {most}")
        bands = None
        sc = rot.get("scaling")
        if sc is not None:
            bands = tuple(float(_get(sc, key, w + "scaling.")) for key in ("factor", "low", "high", "original"))
            if not (bands[0] > 0 and bands[3] > 0 and bands[1] <= bands[2]):
                raise ConfigError(f"{w}scaling: factor and original must be positive and low at most high")
        return RopeHalfAnglesSpec(theta=float(_get(rot, "base", w)), rotary_dim=dims, band_scaling=bands)

    def _mixer(self, layer: Dict[str, Any], where: str):
        w = where + "mixer."
        m = _get(layer, "mixer", where)
        heads, dim, vdim = int(_get(m, "heads", w)), int(_get(m, "dim", w)), int(_get(m, "vdim", w))
        if heads <= 0 or dim <= 0 or vdim <= 0:
            raise ConfigError(f"{w}heads, dim and vdim must be positive")
        if layer["type"] == "hgrn2":
            return ForgetGateLinearSpec(num_heads=heads, head_dim=dim, v_head_dim=vdim, norm_eps=self.eps)
        kv_heads = int(_get(m, "kv_heads", w))
        if kv_heads <= 0 or heads % kv_heads:
            raise ConfigError(f"{w}{heads} heads are no multiple of {kv_heads} key/value heads")
        window = int(_get(m, "mask.size", w))
        if window <= 0:
            raise ConfigError(f"{w}mask.size must be positive")
        cap = float(_get(m, "softcap", w))
        if not cap > 0:
            raise ConfigError(f"{w}softcap must be positive")
        return ConvAttentionSpec(num_heads=heads, num_kv_heads=kv_heads, head_dim=dim, v_head_dim=vdim,
                                 scale=float(_get(m, "scale", w)), qkv_bias=True, out_bias=True, window=window, sink=True,
                                 softcap=cap, position=self._rot(m, w, dim))

    @staticmethod
    def _ffn(layer: Dict[str, Any], where: str):
        mlp = layer.get("mlp")
        if mlp is None:
            return None
        w = where + "mlp."
        kind = _get(mlp, "kind", w)
        if kind != "moe":
            raise ConfigError(f"{w}kind is {kind!r}; known: moe")
        experts, top = int(_get(mlp, "router.experts", w)), int(_get(mlp, "router.top", w))
        ff = int(_get(mlp, "expert.ff", w))
        if not 1 <= top <= experts or ff <= 0:
            raise ConfigError(f"{w}router: top {top} of {experts} experts of width {ff}")
        return SigmoidMoESpec(num_experts=experts, top=top, intermediate_size=ff, weigh_input=True)

    # ---- the model this configuration describes -------------------------------------------------------------------
    def to_model_spec(self) -> ModelSpec:
        norm = BareLayerNormSpec(eps=self.eps)
        conv = ShortConvSpec(taps=self.taps)
        layers = tuple(
            ScaledLayerSpec(prefix=f"l{i}", mixer_norm=norm, mixer=self._mixer(layer, f"layers[{i}]."), ffn_norm=norm,
                            ffn=self._ffn(layer, f"layers[{i}]."), mixer_conv=conv, ffn_conv=conv, layer_scale=True,
                            depth_average=DepthAverageSpec(index=i, layers=len(self.layers)))
            for i, layer in enumerate(self.layers))
        spec = ModelSpec(
            architecture=self.architecture, vocab_size=self.vocab, hidden_size=self.width, layers=layers,
            schedule=tuple(ScheduleEntry(layer=i) for i in range(len(layers))), final_norm=BareLayerNormSpec(eps=self.eps, gain=self.logit_scale),
            embed_name="embed", final_norm_name="final.norm", head_name="head", tie_head=False,
            max_positions=self.max_positions)
        spec.validate()
        return spec
