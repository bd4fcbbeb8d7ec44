"""Host-side tests of the Vuzinex configuration, its model spec, tensor names and cache plan, and of the plain
implementation's mechanisms against library routines and hand sums."""
import copy
import math

import pytest
import torch
import torch.nn.functional as F

import qwen_engine_amd  # noqa: F401
from qwen_engine_amd.cache import GroupSpec
from qwen_engine_amd.config import ConfigError, config_from_dict
from qwen_engine_amd.config.registry import config_from_folder
from qwen_engine_amd.config.spec import RopePairsSpec
from qwen_engine_amd.parts import DecoderModel, Runtime, build_part, cache_plan, expected_tensors
from qwen_engine_amd.weights.random_init import random_tensors
from plain import vuzinex_plain as B
from vuzinex_tiny import TINY, VA, VB, VC, VD, make_folder, random_config, tensor_shapes


@pytest.mark.parametrize("which", sorted(TINY))
def test_expected_tensors_are_the_designs_names(which):
    cfg = TINY[which][0]
    spec = config_from_dict(cfg).to_model_spec()
    want = {k: tuple(v[0]) for k, v in tensor_shapes(cfg).items()}
    assert {k: tuple(v.shape) for k, v in expected_tensors(spec).items()} == want
    assert spec.tie_head and spec.head_name == "embed" and spec.final_norm_name == "final.norm"


def test_spec_and_cache_plan_follow_the_configuration():
    spec = config_from_dict(VA).to_model_spec()
    assert [l.prefix for l in spec.layers] == ["l0", "l1", "l2", "l3"]
    assert [e.layer for e in spec.schedule] == [0, 1, 2, 1, 2, 3] and all(e.cache_from is None for e in spec.schedule)
    assert [l.mixer.kind for l in spec.layers] == ["side_by_side", "state_space", "side_by_side", "state_space"]
    a, r = spec.layers[0].mixer.left, spec.layers[0].mixer.right
    assert (a.num_heads, a.num_kv_heads, a.head_dim, a.v_head_dim, a.chunk, a.scale) == (6, 2, 20, 12, 37, 0.4)
    assert a.head_sink and not a.bias and a.qk_norm is None and not a.output_gate
    assert a.position.band_scaling == (6.0, 1.0, 4.0, 64.0) and a.position.yarn is None and a.position.rotary_dim == 12
    assert (r.kind, r.num_heads, r.head_dim, r.v_head_dim, r.gate_cap) == ("matrix_memory", 3, 12, 20, 9.0)
    assert (spec.layers[0].mixer.left_scale, spec.layers[0].mixer.right_scale) == (1.3, 0.4)
    a, r = spec.layers[2].mixer.left, spec.layers[2].mixer.right
    assert a.chunk is None and a.bias and a.out_bias is False and a.qk_norm == "head" and a.output_gate and not a.head_sink
    assert a.position.yarn == (3.0, 90.0, 8.0, 1.0) and a.position.band_scaling is None
    assert (r.kind, r.decay_rank, r.tau) == ("gated_linear", 9, 5.0)
    m = spec.layers[1].mixer
    assert (m.num_heads, m.head_dim, m.state_dim, m.groups, m.taps, m.norm_groups) == (6, 10, 14, 2, 3, 3)
    assert spec.layers[1].ffn is None and spec.layers[3].ffn.intermediate_size == 56 and spec.layers[3].ffn.bias
    assert all(l.mult == 0.6 and l.mixer_norm.offset == 1.0 for l in spec.layers) and spec.final_norm.gain == 0.7
    pro = spec.stream_prologue
    assert (pro.scale, pro.buckets, pro.mul_prev, pro.mul_cur) == (1.5, 101, 7, 13)
    plan = cache_plan(spec)
    # keys of two layers (one of them twice): all are kept; every run of a layer has a cache or a state of its own; the last
    # user is the embedding's
    assert plan.groups == [GroupSpec(None, 0)] and plan.entry_users == [[i] for i in range(7)]
    assert [k is not None for k in plan.user_kv] == [True, False, True, False, True, False, False]
    up = lambda n: (n + 3) // 4 * 4
    memory = up(3 * 12 * (20 + 1) + 3)                       # matrices, one normaliser (20 columns), running maxima
    ssm = up(up(6 * 14 * 10) + 2 * (60 + 2 * 28))
    assert [s.shape for s in plan.user_state] == [(memory,), (ssm,), (2 * 28 * 16,), (ssm,), (2 * 28 * 16,),
                                                  (up(4 * 20 * 16 + 3 * (64 + 40)),), (1,)]
    assert plan.user_state[6].dtype == "int32"
    # one tap keeps nothing beside the matrices; no loop runs every layer once
    spec = config_from_dict(VC).to_model_spec()
    assert [e.layer for e in spec.schedule] == [0, 1, 2, 3]
    assert cache_plan(spec).user_state[2].shape == (3 * 8 * 8,)
    assert spec.layers[0].mixer.left.position is None and spec.layers[1].mixer.left.position.yarn is None
    assert [e.layer for e in config_from_dict(VB).to_model_spec().schedule] == [0, 1, 0, 1, 0, 1, 2]


def test_two_mixers_side_by_side_share_their_products():
    model = DecoderModel(config_from_dict(VD).to_model_spec())
    assert model.blocks[1].mixer.joint and model.blocks[2].mixer.joint
    kinds = [type(p).__name__ for p in model.all_parts()]
    assert kinds.count("ChunkAttention") == 2 and kinds.count("StateSpaceMixer") == 2      # (also the parts inside others)


def test_the_rank_of_the_decays_comes_from_the_tensors_shape(tmp_path):
    cfg = config_from_folder(make_folder(tmp_path, "A"))
    assert cfg.to_model_spec().layers[2].mixer.right.decay_rank == 9 and cfg.to_dict()["layers"][2]["mixer"]["right"]["decay_rank"] == 9
    d = copy.deepcopy(VA)
    del d["layers"][2]["mixer"]["right"]["decay_rank"]
    with pytest.raises(ConfigError, match="decay_rank"):
        config_from_dict(d)


def test_config_errors_name_the_key():
    for path, message in ((("norm", "eps"), "norm.eps"), (("residual_mult",), "residual_mult"), (("logit_scale",), "logit_scale"),
                          (("embedding", "scale"), "embedding.scale"), (("embedding", "bigram", "buckets"), "embedding.bigram.buckets"),
                          (("embedding", "bigram", "mul_prev"), "mul_prev"), (("loop", "times"), "loop.times"),
                          (("layers", 0, "mixer", "left", "kv_heads"), "layers[0].mixer.left.kv_heads"),
                          (("layers", 0, "mixer", "left", "mask", "size"), "layers[0].mixer.left.mask.size"),
                          (("layers", 0, "mixer", "left", "rot", "scaling", "low"), "layers[0].mixer.left.rot.scaling.low"),
                          (("layers", 0, "mixer", "right", "gate_cap"), "layers[0].mixer.right.gate_cap"),
                          (("layers", 2, "mixer", "left", "rot", "scaling", "fast"), "layers[2].mixer.left.rot.scaling.fast"),
                          (("layers", 2, "mixer", "right", "tau"), "layers[2].mixer.right.tau"),
                          (("layers", 2, "mixer", "right_scale"), "layers[2].mixer.right_scale"),
                          (("layers", 1, "mixer", "norm_groups"), "layers[1].mixer.norm_groups"), (("layers", 3, "mlp", "ff"), "mlp.ff")):
        d = copy.deepcopy(VA)
        cur = d
        for k in path[:-1]:
            cur = cur[k]
        del cur[path[-1]]
        with pytest.raises(ConfigError, match=message.replace("[", r"\[").replace("]", r"\]")):
            config_from_dict(d)
    for change, message in ((lambda d: d["layers"][0]["mixer"]["left"].update(kv_heads=4), "6 heads over 4"),
                            (lambda d: d["layers"][0]["mixer"]["left"]["rot"].update(dims=22), "rot.dims"),
                            (lambda d: d["layers"][0]["mixer"]["left"]["rot"].update(dims=7), "rot.dims"),
                            (lambda d: d["layers"][1]["mixer"].update(groups=4), "4 groups"),
                            (lambda d: d["layers"][1]["mixer"].update(norm_groups=7), "norm_groups"),
                            (lambda d: d["layers"][1]["mixer"].update(state=300), "at most 256"),
                            (lambda d: d["layers"][3]["mlp"].update(kind="moe"), "kind"),
                            (lambda d: d["loop"].update(stop=5), "loop"), (lambda d: d["loop"].update(times=0), "loop"),
                            (lambda d: d["layers"][1].update(type="mamba"), "type")):
        d = copy.deepcopy(VA)
        change(d)
        with pytest.raises(ConfigError, match=message):
            config_from_dict(d)


def test_random_weights_mode_writes_every_tensor():
    got = random_tensors(config_from_dict(VA), seed=5)
    assert {k: tuple(v.shape) for k, v in got.items()} == {k: tuple(v[0]) for k, v in tensor_shapes(VA).items()}
    assert float(got["l0.norm1"].float().abs().max()) < 0.2                 # (stored around zero)


def test_random_configurations_are_read():
    for seed in range(40):
        cfg = random_config(seed)
        spec = config_from_dict(cfg).to_model_spec()
        assert set(expected_tensors(spec)) == set(tensor_shapes(cfg))
        assert [e.layer for e in spec.schedule] == B.layer_order(len(cfg["layers"]), cfg["loop"])


# ---- frequencies ------------------------------------------------------------------------------------------------------
def _freq(**kw):
    part = build_part(RopePairsSpec(**kw), 0)
    part.load({}, Runtime(torch.device("cpu"), torch.float32))
    return part.inv_freq().double(), part.gain


@pytest.mark.parametrize("base,dims,factor,original,fast,slow", [(10000.0, 64, 4.0, 2048, 32.0, 1.0), (500.0, 12, 6.0, 64, 8.0, 1.0),
                                                                 (50.0, 2, 4.0, 30, 4.0, 1.0), (1e6, 128, 32.0, 4096, 32.0, 2.0),
                                                                 (20000.0, 80, 1.5, 100, 1.0, 1.0), (100.0, 40, 2.0, 5, 8.0, 0.1)])
def test_yarn_frequencies(base, dims, factor, original, fast, slow):
    got, gain = _freq(theta=base, rotary_dim=dims, yarn=(factor, float(original), fast, slow))
    want, want_gain = B.yarn(base, dims, dict(factor=factor, original=original, fast=fast, slow=slow))
    want = torch.tensor(want, dtype=torch.float64)
    assert torch.allclose(got, want, rtol=1e-6, atol=0) and abs(gain - want_gain) < 1e-12 and gain > 1.0
    plain = torch.tensor([base ** (-2.0 * i / dims) for i in range(dims // 2)], dtype=torch.float64)
    assert bool((want <= plain * (1 + 1e-12)).all()) and bool((want >= plain / factor * (1 - 1e-12)).all())
    turns = original * plain / (2 * math.pi)
    assert torch.allclose(want[turns > fast * base ** (4.0 / dims)], plain[turns > fast * base ** (4.0 / dims)])


@pytest.mark.parametrize("base,dims,factor,low,high,original", [(10000.0, 64, 8.0, 1.0, 4.0, 8192), (500.0, 12, 6.0, 1.0, 4.0, 64)])
def test_banded_frequencies_of_neighbouring_pairs(base, dims, factor, low, high, original):
    got, gain = _freq(theta=base, rotary_dim=dims, band_scaling=(factor, low, high, float(original)))
    want, _ = B.banded(base, dims, dict(factor=factor, low=low, high=high, original=original))
    assert torch.allclose(got, torch.tensor(want, dtype=torch.float64), rtol=1e-6, atol=0) and gain == 1.0
    assert torch.allclose(_freq(theta=base, rotary_dim=dims)[0], torch.tensor(B.yarn(base, dims, None)[0], dtype=torch.float64), rtol=1e-6)


# ---- the plain implementation's mechanisms against library routines ----------------------------------------------
def _r(g):
    return lambda *s: torch.randn(*s, generator=g, dtype=torch.float64)


def test_plain_norm_gates_and_convolution():
    g = torch.Generator().manual_seed(1)
    r = _r(g)
    x, w = r(9, 48), r(48)
    assert torch.allclose(B.norm_around_one(x, w, 1e-5), F.rms_norm(x, (48,), 1 + w, 1e-5), atol=1e-12)
    z = 30 * r(200)
    assert torch.allclose(B.sigmoid(z), torch.sigmoid(z), atol=1e-14) and torch.allclose(B.silu(z), F.silu(z), atol=1e-12)
    assert torch.allclose(B.log_sigmoid(z), F.logsigmoid(z), atol=1e-12) and torch.allclose(B.softplus(z), F.softplus(z, threshold=1e9), atol=1e-12)
    for taps in (1, 2, 4, 11):
        u, b = r(48, taps), r(48)
        ref = F.conv1d(F.pad(x.t()[None], (taps - 1, 0)), u[:, None, :], b, groups=48)[0].t()
        assert torch.allclose(B.causal_convolution(x, u, b), ref, atol=1e-12)


def test_plain_rows_of_the_second_table():
    assert B.bigram_rows([4, 9, 9, 2], 10, 3, 5) == [10, (12 + 45) % 10, (27 + 45) % 10, (27 + 10) % 10]
    assert B.bigram_rows([7], 1, 3, 5) == [1] and B.layer_order(5, {"start": 1, "stop": 3, "times": 3}) == [0, 1, 2, 1, 2, 1, 2, 3, 4]


def test_plain_rotation_is_a_rotation():
    v = _r(torch.Generator().manual_seed(2))(5, 3, 10)
    pos = torch.tensor([0, 1, 5, 41, 1000])
    freq, gain = B.yarn(100.0, 6, dict(factor=4.0, original=50, fast=8.0, slow=1.0))
    out = B.rotate_neighbours(v, pos, freq, gain)
    assert torch.equal(out[..., 6:], v[..., 6:]) and torch.allclose(out[0, :, :6], gain * v[0, :, :6])
    for i in range(3):
        a = pos.double() * freq[i]
        z = torch.complex(v[..., 2 * i], v[..., 2 * i + 1]) * torch.polar(torch.full_like(a, gain), a)[:, None]
        assert torch.allclose(out[..., 2 * i], z.real, atol=1e-12) and torch.allclose(out[..., 2 * i + 1], z.imag, atol=1e-12)


def test_plain_softmax_with_a_sink():
    r = _r(torch.Generator().manual_seed(3))
    s, seen, sink = 3 * r(4, 7), torch.rand(4, 7, generator=torch.Generator().manual_seed(4)) < 0.7, torch.tensor(1.3, dtype=torch.float64)
    seen[:, 0] = True
    full = torch.cat([s.masked_fill(~seen, -math.inf), sink.expand(4, 1)], dim=1)
    assert torch.allclose(B.softmax_seen(s, seen, sink), torch.softmax(full, dim=1)[:, :-1], atol=1e-12)
    assert torch.allclose(B.softmax_seen(s, seen), torch.softmax(full[:, :-1], dim=1), atol=1e-12)
    assert float(B.softmax_seen(s - 900.0, seen, sink).sum()) == 0.0           # (far below the sink)
    m = B.chunk_mask(7, 3)
    assert m.sum(dim=1).tolist() == [1, 2, 3, 1, 2, 3, 1] and B.chunk_mask(7, None).sum() == 28


def test_plain_recurrences_of_two_tokens_by_hand_and_their_limits():
    r = _r(torch.Generator().manual_seed(5))
    q, k, v = r(2, 2, 3), r(2, 2, 3), r(2, 2, 4)
    alpha = torch.rand(2, 2, 3, generator=torch.Generator().manual_seed(6), dtype=torch.float64)
    o, S = B.decayed_outer(q, k, v, alpha)
    s1 = torch.outer(k[0, 1], v[0, 1])
    s2 = alpha[1, 1][:, None] * s1 + torch.outer(k[1, 1], v[1, 1])
    assert torch.allclose(S[1], s2) and torch.allclose(o[1, 1], s2.t() @ q[1, 1])
    # the matrix memory: without the running maximum (exact while nothing overflows) the same numbers
    i, f = 2 * r(2, 2), F.logsigmoid(2 * r(2, 2))
    o, (S, n, m) = B.matrix_memory(q, k, v, i, f)
    e = torch.exp
    raw = e(f[1, 0]) * e(i[0, 0]) * torch.outer(k[0, 0], v[0, 0]) + e(i[1, 0]) * torch.outer(k[1, 0], v[1, 0])
    n_raw = e(f[1, 0]) * e(i[0, 0]) * k[0, 0] + e(i[1, 0]) * k[1, 0]
    top = max(float(f[1, 0] + max(float(f[0, 0]), float(i[0, 0]))), float(i[1, 0]))
    assert abs(float(m[0]) - top) < 1e-12 and torch.allclose(S[0], raw * math.exp(-top)) and torch.allclose(n[0], n_raw * math.exp(-top))
    den = max(abs(float(n_raw @ q[1, 0])) * math.exp(-top), math.exp(-top)) + 1e-6
    assert torch.allclose(o[1, 0], raw.t() @ q[1, 0] * math.exp(-top) / den)
    assert float(B.matrix_memory(q, k, v, i - 1e3, f)[1][2].max()) <= 0           # the maximum starts at 0, not below every gate
    # the state space: two heads on one group; the skip beside the state's share
    x, dt, A, D = r(2, 2, 4), torch.rand(2, 2, generator=torch.Generator().manual_seed(7), dtype=torch.float64), r(2), r(2)
    y, S = B.state_space(x, k[:, :1], q[:, :1], dt, A, D)
    keep = torch.exp(-torch.exp(A[1]) * dt[1, 1])
    s2 = keep * dt[0, 1] * torch.outer(k[0, 0], x[0, 1]) + dt[1, 1] * torch.outer(k[1, 0], x[1, 1])
    assert torch.allclose(S[1], s2) and torch.allclose(y[1, 1], s2.t() @ q[1, 0] + D[1] * x[1, 1])


def test_plain_gated_feed_forward_with_biases():
    r = _r(torch.Generator().manual_seed(8))
    w = {"gate": r(5, 6), "gate.b": r(5), "up": r(5, 6), "up.b": r(5), "down": r(6, 5), "down.b": r(6)}
    h = r(3, 6)
    ref = F.linear(F.silu(F.linear(h, w["gate"], w["gate.b"])) * F.linear(h, w["up"], w["up.b"]), w["down"], w["down.b"])
    assert torch.allclose(B.gated_mlp(h, w, ""), ref, atol=1e-12)
