"""Mixers that carry a matrix per head from token to token instead of keys and values, and the mixer that runs
two mixers side by side.  A request's state lives in its state slot, in 32-bit, and is cleared when the request
starts; a portion cut anywhere continues where the last one ended."""
from __future__ import annotations

from typing import Dict, Optional

import torch

from ..cache.plan import StateNeed
from ..kernels import ops
from .base import CacheBinding, Runtime, TensorInfo, join_name, named_tensors
from .projected import InputProducts, OutputProduct, ProjectedMixer
from .registry import build_part, part_class, register_part


# From this many rows of one request in a step, the recurrences take the step's rows chunk by chunk (the chunks in
# parallel) instead of row by row.
CHUNKED_FROM_ROWS = 8


def _chunks(ctx, heads: int, v_dim: int = 128):
    """The step's rows cut into chunks for the chunked recurrence, if a request brings many rows: built and sent to the
    device once per step and chunk length, shared by the layers.  ``v_dim``: value columns a head, where the decays are given
    (the kernels then run blocks of four waves up to 64).  None: row by row."""
    longest = max((s.q_len for s in ctx.seqs), default=0)
    if longest < CHUNKED_FROM_ROWS:
        return None
    C = ops.recurrence_chunk_len(longest, heads, small_blocks=v_dim <= 64)
    key = ("recurrence.chunks", C)
    if key not in ctx.memo:
        ch, po = ops.recurrence_chunks([(s.q_start, s.q_len) for s in ctx.seqs], C)
        ctx.memo[key] = (ch.to(ctx.rt.device), po.to(ctx.rt.device))
    return ctx.memo[key]


class ShiftedDecayMixer:
    """``ShiftedDecaySpec``: five blends of each token with the token before it, projections r, k, v, a silu gate
    and a decay per key channel through a low rank, the recurrence with a bonus for the token itself, a norm per
    head, the gate, the output projection.  State: the request's last input row, then the heads' matrices."""
    graph_safe = True
    BLENDS = ("r", "k", "v", "g", "w")

    def __init__(self, spec, hidden_size: int):
        self.spec = spec
        self.hidden = int(hidden_size)
        self.h, self.d, self.rank = int(spec.num_heads), int(spec.head_dim), int(spec.decay_rank)
        self.eps = float(spec.norm_eps)
        self.mu = self.w_r = self.w_k = self.w_v = self.w_g = self.w_1 = self.w_2 = self.w_o = None
        self.w0 = self.u = self.norm = None

    @staticmethod
    def expected_tensors(spec, hidden: int) -> Dict[str, TensorInfo]:
        n = spec.num_heads * spec.head_dim
        t = {f"mu.{s}": TensorInfo((hidden,), "normal", "vector") for s in ShiftedDecayMixer.BLENDS}
        for name in ("r", "k", "v", "g"):
            t[name] = TensorInfo((n, hidden))
        t["w1"] = TensorInfo((int(spec.decay_rank), hidden))
        t["w2"] = TensorInfo((n, int(spec.decay_rank)))
        t["w0"] = TensorInfo((n,), "zeros", "vector")
        t["u"] = TensorInfo((spec.num_heads, spec.head_dim), "normal", "vector")
        t["norm"] = TensorInfo((n,), "ones", "vector")
        t["o"] = TensorInfo((hidden, n))
        return t

    @staticmethod
    def cache_need(spec):
        return None

    @staticmethod
    def state_need(spec, hidden: int) -> Optional[StateNeed]:
        return StateNeed(shape=(hidden + spec.num_heads * spec.head_dim * spec.head_dim,), dtype="float32")

    def load(self, tensors: Dict[str, torch.Tensor], rt: Runtime) -> None:
        self.mu = rt.place_vector(torch.stack([tensors[f"mu.{s}"].float() for s in self.BLENDS]))
        self.w_r, self.w_k, self.w_v, self.w_g = (rt.place_matrix(tensors[n]) for n in ("r", "k", "v", "g"))
        self.w_1, self.w_2, self.w_o = (rt.place_matrix(tensors[n]) for n in ("w1", "w2", "o"))
        self.w0 = rt.place_vector(tensors["w0"])
        self.u = rt.place_vector(tensors["u"].reshape(-1))
        self.norm = rt.place_vector(tensors["norm"])

    def forward(self, x: torch.Tensor, ctx, binding: CacheBinding) -> torch.Tensor:
        if binding.state is None:
            raise RuntimeError("the recurrence was given no state")
        T, W, st = x.shape[0], self.hidden, binding.state
        m = ops.token_shift(x, self.mu, st, ctx.tok_seq, single_rows=ctx.single_rows)
        r, k, v, gate = (ops.gemm(m[i], w) for i, w in enumerate((self.w_r, self.w_k, self.w_v, self.w_g)))
        low = ops.unary(ops.gemm(m[4], self.w_1, out_dtype=torch.float32), ops.UNARY_TANH, out_dtype=ctx.rt.dtype)
        decay_x = ops.gemm(low, self.w_2, out_dtype=torch.float32)      # (exponentials of the decay: in the recurrence, 32-bit)
        o = ops.linear_recurrence(r, k, v, st[:, W:], ctx.tok_seq, self.h, decay_x=decay_x, decay_bias=self.w0,
                                  bonus=self.u, chunks=_chunks(ctx, self.h))
        y = ops.gated_norm(o.view(T, self.h * self.d), self.norm, self.eps, self.h, ctx.rt.dtype, gate=gate,
                           gate_act=ops.GATE_SILU)
        return ops.gemm(y, self.w_o, out_dtype=torch.float32)


class DecayedLinearMixer:
    """``DecayedLinearSpec``: one product for q | k | v | gate, the recurrence with one decay per head (silu on q, k
    and v as they are read), all heads normed together, the sigmoid gate, the output projection."""
    graph_safe = True

    def __init__(self, spec, hidden_size: int):
        self.spec = spec
        self.hidden = int(hidden_size)
        self.h, self.d, self.dv = int(spec.num_heads), int(spec.head_dim), int(spec.v_head_dim)
        if len(spec.decay) != self.h:
            raise ValueError(f"{len(spec.decay)} decays for {self.h} heads")
        self.eps = float(spec.norm_eps)
        self.w_in = self.w_o = self.norm = self.decay = None

    @staticmethod
    def expected_tensors(spec, hidden: int) -> Dict[str, TensorInfo]:
        nk, nv = spec.num_heads * spec.head_dim, spec.num_heads * spec.v_head_dim
        return {"q": TensorInfo((nk, hidden)), "k": TensorInfo((nk, hidden)), "v": TensorInfo((nv, hidden)),
                "g": TensorInfo((nv, hidden)), "o": TensorInfo((hidden, nv)), "norm": TensorInfo((nv,), "ones", "vector")}

    @staticmethod
    def cache_need(spec):
        return None

    @staticmethod
    def state_need(spec, hidden: int) -> Optional[StateNeed]:
        return StateNeed(shape=(spec.num_heads * spec.head_dim * spec.v_head_dim,), dtype="float32")

    def load(self, tensors: Dict[str, torch.Tensor], rt: Runtime) -> None:
        mats = [tensors[n] for n in ("q", "k", "v", "g")]
        if len({m.dtype for m in mats}) > 1:
            mats = [m.float() for m in mats]
        self.w_in = rt.place_matrix(torch.cat(mats, dim=0))
        self.w_o = rt.place_matrix(tensors["o"])
        self.norm = rt.place_vector(tensors["norm"])
        self.decay = torch.tensor(list(self.spec.decay), dtype=torch.float64).to(torch.float32).to(rt.device)

    def forward(self, x: torch.Tensor, ctx, binding: CacheBinding) -> torch.Tensor:
        if binding.state is None:
            raise RuntimeError("the recurrence was given no state")
        T = x.shape[0]
        nk, nv = self.h * self.d, self.h * self.dv
        y = ops.gemm(x, self.w_in)
        o = ops.linear_recurrence(y[:, :nk], y[:, nk:2 * nk], y[:, 2 * nk:2 * nk + nv], binding.state, ctx.tok_seq,
                                  self.h, decay=self.decay, silu=True, chunks=_chunks(ctx, self.h))
        z = ops.gated_norm(o.view(T, nv), self.norm, self.eps, 1, ctx.rt.dtype, gate=y[:, 2 * nk + nv:],
                           gate_act=ops.GATE_SIGMOID)
        return ops.gemm(z, self.w_o, out_dtype=torch.float32)


class ForgetGateLinearMixer:
    """``ForgetGateLinearSpec`` (HGRN2): one product for q | f | v that stays 32-bit (the gate enters the recurrence), the
    recurrence (silu on q, the gate and what it leaves to be written formed as they are read) with the norm per head
    behind it (one launch for single new tokens), the output projection."""
    graph_safe = True

    def __init__(self, spec, hidden_size: int):
        self.spec = spec
        self.hidden = int(hidden_size)
        self.h, self.d, self.dv = int(spec.num_heads), int(spec.head_dim), int(spec.v_head_dim)
        self.eps = float(spec.norm_eps)
        self.w_in = self.w_o = self.norm = self.forget_bias = self.lower = None

    @staticmethod
    def expected_tensors(spec, hidden: int) -> Dict[str, TensorInfo]:
        nk, nv = spec.num_heads * spec.head_dim, spec.num_heads * spec.v_head_dim
        q, f, fb, low, v, norm, o = spec.names
        return {q: TensorInfo((nk, hidden)), f: TensorInfo((nk, hidden)), fb: TensorInfo((nk,), "zeros", "vector"),
                low: TensorInfo((nk,), "zeros", "vector"), v: TensorInfo((nv, hidden)),
                norm: TensorInfo((int(spec.v_head_dim),), "ones", "vector"), o: TensorInfo((hidden, nv))}

    @staticmethod
    def cache_need(spec):
        return None

    @staticmethod
    def state_need(spec, hidden: int) -> Optional[StateNeed]:
        return StateNeed(shape=(spec.num_heads * spec.head_dim * spec.v_head_dim,), dtype="float32")

    def load(self, tensors: Dict[str, torch.Tensor], rt: Runtime) -> None:
        q, f, fb, low, v, norm, o = self.spec.names
        mats = [tensors[n] for n in (q, f, v)]
        if len({m.dtype for m in mats}) > 1:
            mats = [m.float() for m in mats]
        self.w_in = rt.place_matrix(torch.cat(mats, dim=0))
        self.w_o = rt.place_matrix(tensors[o])
        self.forget_bias = rt.place_vector(tensors[fb])
        self.lower = rt.place_vector(tensors[low])
        self.norm = rt.place_vector(tensors[norm]).repeat(self.h)

    def forward(self, x: torch.Tensor, ctx, binding: CacheBinding) -> torch.Tensor:
        if binding.state is None:
            raise RuntimeError("the recurrence was given no state")
        T = x.shape[0]
        nk = self.h * self.d
        y = ops.gemm(x, self.w_in, out_dtype=torch.float32)
        z = ops.linear_recurrence(y[:, :nk], y[:, nk:2 * nk], y[:, 2 * nk:], binding.state, ctx.tok_seq, self.h, silu=True,
                                  forget_bias=self.forget_bias, lower=self.lower, chunks=_chunks(ctx, self.h),
                                  norm_weight=self.norm, norm_eps=self.eps, norm_dtype=ctx.rt.dtype,
                                  single_rows=ctx.single_rows)
        splits = ops.gemm_branch_splits(z, self.w_o)
        if splits:
            return ops.gemm(z, self.w_o, epilogue=ops.EPI_PARTIAL, splits=splits)
        return ops.gemm(z, self.w_o)


class GatedLinearMixer(ProjectedMixer):
    """``GatedLinearSpec``: the decays come from the low-rank projection in a kernel of their own (single new tokens: inside the
    recurrence), the recurrence has the norm per head and the silu gate behind it."""

    def __init__(self, spec, hidden_size: int):
        self.spec = spec
        self.hidden = int(hidden_size)
        self.h, self.d, self.dv, self.rank = int(spec.num_heads), int(spec.head_dim), int(spec.v_head_dim), int(spec.decay_rank)
        self.tau, self.eps = float(spec.tau), float(spec.norm_eps)
        self.w_2 = self.b_2 = self.norm = None

    @staticmethod
    def expected_tensors(spec, hidden: int) -> Dict[str, TensorInfo]:
        nk, nv = spec.num_heads * spec.head_dim, spec.num_heads * spec.v_head_dim
        q, k, v, g, o, norm, a1, a2, a2b = spec.names
        return {q: TensorInfo((nk, hidden)), k: TensorInfo((nk, hidden)), v: TensorInfo((nv, hidden)), g: TensorInfo((nv, hidden)),
                o: TensorInfo((hidden, nv)), norm: TensorInfo((int(spec.v_head_dim),), "ones", "vector"),
                a1: TensorInfo((int(spec.decay_rank), hidden)), a2: TensorInfo((nk, int(spec.decay_rank))),
                a2b: TensorInfo((nk,), "zeros", "vector")}

    @staticmethod
    def cache_need(spec):
        return None

    @staticmethod
    def state_need(spec, hidden: int) -> Optional[StateNeed]:
        return StateNeed(shape=(ops.recurrence_state_numbers(spec.num_heads, spec.head_dim, spec.v_head_dim),), dtype="float32")

    def inputs(self, tensors):
        q, k, v, g, _, _, a1, _, _ = self.spec.names
        return [(tensors[n], None) for n in (q, k, v, g, a1)], []

    def output(self, tensors):
        return tensors[self.spec.names[4]]

    def load_own(self, tensors: Dict[str, torch.Tensor], rt: Runtime) -> None:
        _, _, _, _, _, norm, _, a2, a2b = self.spec.names
        self.w_2 = rt.place_vector(tensors[a2].t())          # [rank, channels], 32-bit: neighbouring channels side by side
        self.b_2 = rt.place_vector(tensors[a2b])
        self.norm = rt.place_vector(tensors[norm]).repeat(self.h)

    def mix(self, y: torch.Tensor, gates, ctx, binding: CacheBinding, out: torch.Tensor, factor: float = 1.0) -> None:
        if binding.state is None:
            raise RuntimeError("the recurrence was given no state")
        nk, nv = self.h * self.d, self.h * self.dv
        ops.linear_recurrence(y[:, :nk], y[:, nk:2 * nk], y[:, 2 * nk:2 * nk + nv], binding.state, ctx.tok_seq, self.h,
                              low_rank=(y[:, 2 * nk + 2 * nv:], self.w_2, self.b_2, self.tau), q_scale=self.d ** -0.5,
                              chunks=_chunks(ctx, self.h, self.dv), norm_weight=self.norm, norm_eps=self.eps, norm_dtype=ctx.rt.dtype,
                              single_rows=ctx.single_rows, gate=y[:, 2 * nk + nv:2 * nk + 2 * nv], gate_act=ops.GATE_SILU,
                              y_scale=factor, out=out)


class MatrixMemoryMixer(ProjectedMixer):
    """``MatrixMemorySpec``: the two gates' logits stay 32-bit; a kernel turns them into decays, key factors and floors
    along the running maximum (single new tokens: inside the recurrence); the recurrence carries its normaliser and has the
    norm per head and the sigmoid gate behind it.  State: the matrices, the normalisers, the running maxima."""

    def __init__(self, spec, hidden_size: int):
        self.spec = spec
        self.hidden = int(hidden_size)
        self.h, self.d, self.dv = int(spec.num_heads), int(spec.head_dim), int(spec.v_head_dim)
        self.cap, self.eps = float(spec.gate_cap), float(spec.norm_eps)
        self.b_i = self.b_f = self.norm = None

    @staticmethod
    def expected_tensors(spec, hidden: int) -> Dict[str, TensorInfo]:
        h, nk, nv = spec.num_heads, spec.num_heads * spec.head_dim, spec.num_heads * spec.v_head_dim
        q, k, v, g, o, norm, i, ib, f, fb = spec.names
        return {q: TensorInfo((nk, hidden)), k: TensorInfo((nk, hidden)), v: TensorInfo((nv, hidden)), g: TensorInfo((nv, hidden)),
                o: TensorInfo((hidden, nv)), norm: TensorInfo((nv,), "ones", "vector"),
                i: TensorInfo((h, hidden)), ib: TensorInfo((h,), "zeros", "vector"),
                f: TensorInfo((h, hidden)), fb: TensorInfo((h,), "zeros", "vector")}

    @staticmethod
    def cache_need(spec):
        return None

    @staticmethod
    def state_need(spec, hidden: int) -> Optional[StateNeed]:
        n = ops.recurrence_state_numbers(spec.num_heads, spec.head_dim, spec.v_head_dim, normaliser=True) + spec.num_heads
        return StateNeed(shape=((n + 3) // 4 * 4,), dtype="float32")        # (rows of whole 16-byte pieces)

    def inputs(self, tensors):
        q, k, v, g, _, _, i, _, f, _ = self.spec.names
        return [(tensors[n], None) for n in (q, k, v, g)], [tensors[i], tensors[f]]

    def output(self, tensors):
        return tensors[self.spec.names[4]]

    def load_own(self, tensors: Dict[str, torch.Tensor], rt: Runtime) -> None:
        self.norm, self.b_i, self.b_f = (rt.place_vector(tensors[self.spec.names[n]]) for n in (5, 7, 9))

    def mix(self, y: torch.Tensor, gates, ctx, binding: CacheBinding, out: torch.Tensor, factor: float = 1.0) -> None:
        st = binding.state
        if st is None:
            raise RuntimeError("the recurrence was given no state")
        nk, nv = self.h * self.d, self.h * self.dv
        at = ops.recurrence_state_numbers(self.h, self.d, self.dv, normaliser=True)
        ops.linear_recurrence(y[:, :nk], y[:, nk:2 * nk], y[:, 2 * nk:2 * nk + nv], st, ctx.tok_seq, self.h,
                              gates=(gates, self.b_i, self.b_f, self.cap, at), q_scale=self.d ** -0.5,
                              chunks=_chunks(ctx, self.h, self.dv), norm_weight=self.norm, norm_eps=self.eps, norm_dtype=ctx.rt.dtype,
                              single_rows=ctx.single_rows, gate=y[:, 2 * nk + nv:], gate_act=ops.GATE_SIGMOID, y_scale=factor,
                              out=out)


class StateSpaceMixer(ProjectedMixer):
    """``StateSpaceSpec`` (Mamba-2): the step sizes' logits stay 32-bit; one kernel convolves x, B and C and forms step sizes and
    decays, the recurrence runs over them (its keys scaled by the step sizes), one kernel adds the skip, gates and norms.
    State: the heads' matrices, the convolution's last inputs."""

    def __init__(self, spec, hidden_size: int):
        self.spec = spec
        self.hidden = int(hidden_size)
        self.h, self.dv, self.n, self.groups = int(spec.num_heads), int(spec.head_dim), int(spec.state_dim), int(spec.groups)
        self.taps, self.norm_groups, self.eps = int(spec.taps), int(spec.norm_groups), float(spec.norm_eps)
        self.conv_w_t = self.conv_b = self.dt_bias = self.a_log = self.skip = self.norm = None

    @staticmethod
    def _sizes(spec):
        """(inner, convolved channels)."""
        inner = spec.num_heads * spec.head_dim
        return inner, inner + 2 * spec.groups * spec.state_dim

    @staticmethod
    def expected_tensors(spec, hidden: int) -> Dict[str, TensorInfo]:
        inner, C = StateSpaceMixer._sizes(spec)
        w_in, conv, conv_b, dt_b, a_log, skip, norm, o = spec.names
        h = spec.num_heads
        return {w_in: TensorInfo((inner + C + h, hidden)), conv: TensorInfo((C, int(spec.taps)), "normal", "vector"),
                conv_b: TensorInfo((C,), "zeros", "vector"), dt_b: TensorInfo((h,), "zeros", "vector"),
                a_log: TensorInfo((h,), "zeros", "vector"), skip: TensorInfo((h,), "ones", "vector"),
                norm: TensorInfo((inner,), "ones", "vector"), o: TensorInfo((hidden, inner))}

    @staticmethod
    def cache_need(spec):
        return None

    @staticmethod
    def _state_offset(spec) -> int:
        """Where the convolution's inputs begin in a state row (behind the matrices, at a whole 16-byte piece)."""
        return (ops.recurrence_state_numbers(spec.num_heads, spec.state_dim, spec.head_dim) + 3) // 4 * 4

    @staticmethod
    def state_need(spec, hidden: int) -> Optional[StateNeed]:
        n = StateSpaceMixer._state_offset(spec) + (int(spec.taps) - 1) * StateSpaceMixer._sizes(spec)[1]
        return StateNeed(shape=((n + 3) // 4 * 4,), dtype="float32")

    def inputs(self, tensors):
        inner, C = self._sizes(self.spec)
        w = tensors[self.spec.names[0]]
        return [(w[:inner + C], None)], [w[inner + C:]]

    def output(self, tensors):
        return tensors[self.spec.names[7]]

    def load_own(self, tensors: Dict[str, torch.Tensor], rt: Runtime) -> None:
        _, conv, conv_b, dt_b, a_log, skip, norm, _ = self.spec.names
        self.conv_w_t = rt.place_vector(tensors[conv].t())
        self.conv_b, self.dt_bias, self.a_log, self.skip, self.norm = (rt.place_vector(tensors[n])
                                                                       for n in (conv_b, dt_b, a_log, skip, norm))

    def mix(self, y: torch.Tensor, gates, ctx, binding: CacheBinding, out: torch.Tensor, factor: float = 1.0) -> None:
        st = binding.state
        if st is None:
            raise RuntimeError("the recurrence was given no state")
        if factor != 1.0:
            raise ValueError("the state space leaves its result as it is")
        inner, C = self._sizes(self.spec)
        gn = self.groups * self.n
        chunks = _chunks(ctx, self.h, self.dv)
        xbc, steps = ops.conv_steps(y[:, inner:], self.conv_w_t, self.conv_b, st[:, self._state_offset(self.spec):], ctx.tok_seq,
                                    dt=gates, dt_bias=self.dt_bias, a_log=self.a_log, single_rows=ctx.single_rows, chunks=chunks)
        x = xbc[:, :inner]
        o = ops.linear_recurrence(xbc[:, inner + gn:], xbc[:, inner:inner + gn], x, st, ctx.tok_seq, self.h, steps=steps,
                                  k_heads=self.groups, chunks=chunks, single_rows=ctx.single_rows)
        ops.skip_gate_norm(o, x, self.skip, y[:, :inner], self.norm, self.eps, self.norm_groups, ctx.rt.dtype, out=out)


class SideBySideMixer:
    """``SideBySideMixerSpec``: two mixers read the same rows; their outputs are added with weights, in 32-bit.  The
    two share the block's one cache binding: the keys and values of the one that has any, the state of the one that
    has any.  Two projected mixers (parts.projected) share the products before and behind them: what they leave lies side by
    side in one row, the right one's part times right_scale / left_scale, and left_scale goes to whoever adds the result."""

    def __init__(self, spec, hidden_size: int):
        self.spec = spec
        self.hidden = int(hidden_size)
        self.left = build_part(spec.left, hidden_size)
        self.right = build_part(spec.right, hidden_size)
        self.left_scale, self.right_scale = float(spec.left_scale), float(spec.right_scale)
        self.joint = self.left_scale != 0.0 and self._projected(spec.left) and self._projected(spec.right) and \
            isinstance(self.right, (GatedLinearMixer, MatrixMemoryMixer))
        self.products_in: Optional[InputProducts] = None
        self.products_out: Optional[OutputProduct] = None

    @staticmethod
    def _projected(spec) -> bool:
        cls = part_class(spec.kind)
        return cls.is_projected(spec) if hasattr(cls, "is_projected") else issubclass(cls, ProjectedMixer)

    def parts(self):
        return (self.left, self.right)

    @property
    def graph_safe(self):
        return getattr(self.left, "graph_safe", False) is True and getattr(self.right, "graph_safe", False) is True

    @staticmethod
    def _subs(spec):
        return list(zip(spec.names, (spec.left, spec.right)))

    @staticmethod
    def expected_tensors(spec, hidden: int) -> Dict[str, TensorInfo]:
        out: Dict[str, TensorInfo] = {}
        for name, sub in SideBySideMixer._subs(spec):
            for rel, info in part_class(sub.kind).expected_tensors(sub, hidden).items():
                out[join_name(name, rel)] = info
        return out

    @staticmethod
    def _one(spec, hidden, what: str):
        found = []
        for _, sub in SideBySideMixer._subs(spec):
            cls = part_class(sub.kind)
            if hasattr(cls, what):
                need = getattr(cls, what)(sub) if what == "cache_need" else getattr(cls, what)(sub, hidden)
                if need is not None:
                    found.append(need)
        if len(found) > 1:
            raise ValueError(f"two mixers side by side both ask for a {what.split('_')[0]}: one binding holds one")
        return found[0] if found else None

    @staticmethod
    def cache_need(spec):
        return SideBySideMixer._one(spec, 0, "cache_need")

    @staticmethod
    def state_need(spec, hidden: int):
        return SideBySideMixer._one(spec, hidden, "state_need")

    def load(self, tensors: Dict[str, torch.Tensor], rt: Runtime) -> None:
        held = [named_tensors(tensors, name, type(part).expected_tensors(sub, self.hidden))
                for (name, sub), part in zip(self._subs(self.spec), (self.left, self.right))]
        both = list(zip((self.left, self.right), held))
        if not self.joint:
            for part, t in both:
                part.load(t, rt)
            return
        for part, t in both:
            part.load_own(t, rt)
        self.products_in = InputProducts([part.inputs(t) for part, t in both], rt)
        self.products_out = OutputProduct([part.output(t) for part, t in both], rt)

    def forward_scaled(self, x: torch.Tensor, ctx, binding: CacheBinding):
        """(y, s): the output is s * y, y [T, H] or float32 partial products [S, T, H]."""
        if not self.joint:
            return self.forward(x, ctx, binding), 1.0
        ins = self.products_in.run(x, ctx.rt)
        o = self.products_out.rows(x.shape[0], ctx.rt, x.device)
        for part, (y, gates), (a, b), factor in zip((self.left, self.right), ins, self.products_out.cols,
                                                    (1.0, self.right_scale / self.left_scale)):
            part.mix(y, gates, ctx, binding, o[:, a:b], factor)
        return self.products_out.run(o), self.left_scale

    def forward(self, x: torch.Tensor, ctx, binding: CacheBinding) -> torch.Tensor:
        if self.joint:
            y, scale = self.forward_scaled(x, ctx, binding)
            return y if scale == 1.0 else ops.scaled_sum(y, scale, y, 0.0)
        a, b = (part.forward(x, ctx, binding) for part in (self.left, self.right))
        if a.dtype != b.dtype or a.shape != b.shape:
            a, b = (t.float().sum(0) if t.dim() == 3 else t.float() for t in (a, b))
        return ops.scaled_sum(a, self.left_scale, b, self.right_scale)


register_part("gated_linear", GatedLinearMixer)
register_part("matrix_memory", MatrixMemoryMixer)
register_part("state_space", StateSpaceMixer)
register_part("shifted_decay", ShiftedDecayMixer)
register_part("decayed_linear", DecayedLinearMixer)
register_part("forget_gate_linear", ForgetGateLinearMixer)
register_part("side_by_side", SideBySideMixer)
