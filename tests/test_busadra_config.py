"""Host-side tests of the Busadra configuration, its model spec, tensor names and cache plan, and of the plain
implementation's mechanisms against library routines and hand sums."""
import copy
import math

import pytest
import torch
import torch.nn.functional as F

import qwen_engine_amd  # noqa: F401
from qwen_engine_amd.cache import GroupSpec
from qwen_engine_amd.config import ConfigError, config_from_dict
from qwen_engine_amd.config.spec import RopeHalfAnglesSpec
from qwen_engine_amd.parts import Runtime, build_part, cache_plan, expected_tensors
from qwen_engine_amd.weights.random_init import random_tensors
from plain import busadra_plain as B
from busadra_tiny import BA, BC, BD, TINY, random_config, tensor_shapes


@pytest.mark.parametrize("which", sorted(TINY))
def test_expected_tensors_are_the_designs_names(which):
    cfg = TINY[which][0]
    spec = config_from_dict(cfg).to_model_spec()
    want = {k: tuple(v[0]) for k, v in tensor_shapes(cfg).items()}
    expected = expected_tensors(spec)
    assert {k: tuple(v.shape) for k, v in expected.items() if not v.optional} == want
    # what stands around a feed-forward that is not there may be in the folder, and nothing else
    extra = {k for k, v in expected.items() if v.optional}
    assert extra == {f"l{i}.{n}" for i, l in enumerate(cfg["layers"]) if l["mlp"] is None for n in ("norm2", "canon2", "ls2")}
    assert not spec.tie_head and spec.head_name == "head" and spec.final_norm_name == "final.norm"


def test_spec_and_cache_plan_follow_the_configuration():
    spec = config_from_dict(BA).to_model_spec()
    assert [l.prefix for l in spec.layers] == ["l0", "l1", "l2", "l3"]
    assert [l.mixer.kind for l in spec.layers] == ["conv_attention", "forget_gate_linear", "forget_gate_linear", "conv_attention"]
    m = spec.layers[0].mixer
    assert (m.num_heads, m.num_kv_heads, m.head_dim, m.v_head_dim, m.window, m.scale, m.softcap) == (6, 2, 20, 12, 37, 0.4, 4.0)
    assert m.sink and m.qkv_bias and m.out_bias and m.conv_taps == 0 and m.keep_first == 0
    assert m.position.rotary_dim == 12 and m.position.theta == 500.0 and m.position.band_scaling == (6.0, 1.0, 4.0, 64.0)
    r = spec.layers[2].mixer
    assert (r.num_heads, r.head_dim, r.v_head_dim, r.norm_eps) == (2, 28, 16, 1e-6)
    assert spec.layers[1].ffn is None
    f = spec.layers[2].ffn
    assert (f.kind, f.num_experts, f.top, f.intermediate_size, f.weigh_input, f.router_bias) == ("sigmoid_moe", 5, 3, 24, True, False)
    assert all(l.layer_scale and l.mixer_conv.taps == 3 and l.ffn_conv.taps == 3 for l in spec.layers)
    assert [(l.depth_average.index, l.depth_average.layers) for l in spec.layers] == [(0, 4), (1, 4), (2, 4), (3, 4)]
    assert spec.final_norm.gain == 0.7 and spec.layers[0].mixer_norm.gain == 1.0
    assert config_from_dict(BC).to_model_spec().layers[0].mixer.position.band_scaling is None
    plan = cache_plan(spec)
    assert plan.groups == [GroupSpec(37, 0), GroupSpec(9, 0)]
    # per layer: the mixer, then the convolution of each sublayer there is
    assert [len(u) for u in plan.entry_users] == [3, 2, 3, 3]
    shapes = [None if s is None else s.shape for s in plan.user_state]
    assert shapes == [None, (2, 96), (2, 96), (3 * 12 * 20,), (2, 96), (2 * 28 * 16,), (2, 96), (2, 96), None, (2, 96), (2, 96)]
    # one tap keeps nothing
    plan = cache_plan(config_from_dict(BC).to_model_spec())
    assert [s.shape for s in plan.user_state if s is not None] == [(16 * 8,)]


def test_config_errors_name_the_key():
    for path, message in ((("norm", "eps"), "norm.eps"), (("canon", "taps"), "canon.taps"), (("logit_scale",), "logit_scale"),
                          (("layers", 0, "mixer", "kv_heads"), "layers[0].mixer.kv_heads"),
                          (("layers", 0, "mixer", "softcap"), "layers[0].mixer.softcap"),
                          (("layers", 0, "mixer", "mask", "size"), "layers[0].mixer.mask.size"),
                          (("layers", 3, "mixer", "rot", "scaling", "high"), "layers[3].mixer.rot.scaling.high"),
                          (("layers", 1, "mixer", "vdim"), "layers[1].mixer.vdim"),
                          (("layers", 2, "mlp", "router", "top"), "router.top"), (("layers", 2, "mlp", "expert", "ff"), "expert.ff")):
        d = copy.deepcopy(BA)
        cur = d
        for k in path[:-1]:
            cur = cur[k]
        del cur[path[-1]]
        with pytest.raises(ConfigError, match=message.replace("[", r"\[").replace("]", r"\]")):
            config_from_dict(d)
    for change, message in ((lambda d: d["layers"][0]["mixer"].update(kv_heads=4), "multiple"),
                            (lambda d: d["layers"][0]["mixer"]["rot"].update(dims=22), "rot.dims"),
                            (lambda d: d["layers"][0]["mixer"]["rot"].update(dims=7), "rot.dims"),
                            (lambda d: d["layers"][2]["mlp"]["router"].update(top=6), "top 6 of 5"),
                            (lambda d: d["layers"][2]["mlp"].update(kind="dense"), "kind"),
                            (lambda d: d["canon"].update(taps=0), "taps"),
                            (lambda d: d["layers"][1].update(type="gla"), "type")):
        d = copy.deepcopy(BA)
        change(d)
        with pytest.raises(ConfigError, match=message):
            config_from_dict(d)


def test_random_weights_mode_writes_every_tensor():
    got = random_tensors(config_from_dict(BA), seed=5)
    want = {k: tuple(v[0]) for k, v in tensor_shapes(BA).items()}
    assert {k: tuple(got[k].shape) for k in want} == want


def test_random_configurations_are_read():
    for seed in range(40):
        cfg = random_config(seed)
        spec = config_from_dict(cfg).to_model_spec()
        assert {k for k, v in expected_tensors(spec).items() if not v.optional} == set(tensor_shapes(cfg))


# ---- frequencies by bands of wavelengths ------------------------------------------------------------------------------
@pytest.mark.parametrize("base,dims,factor,low,high,original", [(10000.0, 64, 8.0, 1.0, 4.0, 8192), (500.0, 12, 6.0, 1.0, 4.0, 64),
                                                                (100.0, 8, 3.0, 2.0, 2.0, 100), (1e6, 128, 32.0, 0.5, 16.0, 2048),
                                                                (300.0, 6, 1.0, 1.0, 8.0, 40)])
def test_banded_frequencies(base, dims, factor, low, high, original):
    part = build_part(RopeHalfAnglesSpec(theta=base, rotary_dim=dims, band_scaling=(factor, low, high, float(original))), 0)
    part.load({}, Runtime(torch.device("cpu"), torch.float32))
    want = torch.tensor(B.frequencies(base, dims, dict(factor=factor, low=low, high=high, original=original)), dtype=torch.float64)
    assert torch.allclose(part.inv_freq().double(), want, rtol=1e-6, atol=0)
    plain = torch.tensor([base ** (-2.0 * i / dims) for i in range(dims // 2)], dtype=torch.float64)
    turns = original * plain / (2 * math.pi)
    assert torch.allclose(want[turns > high], plain[turns > high]) and torch.allclose(want[turns < low], plain[turns < low] / factor)
    if high > low:
        mid = (turns > low) & (turns < high)
        assert bool(((want[mid] <= plain[mid]) & (want[mid] >= plain[mid] / factor)).all())


# ---- the plain implementation's mechanisms against library routines ----------------------------------------------
def test_plain_norms_and_convolution():
    g = torch.Generator().manual_seed(1)
    x = torch.randn(9, 48, generator=g, dtype=torch.float64) + 0.7
    w = torch.randn(48, generator=g, dtype=torch.float64)
    assert torch.allclose(B.layer_norm(x, w, 1e-5), F.layer_norm(x, (48,), w, None, 1e-5), atol=1e-12)
    assert torch.allclose(B.rms_norm(x, w, 1e-5), F.rms_norm(x, (48,), w, 1e-5), atol=1e-12)
    for taps in (1, 2, 4, 11):
        u = torch.randn(48, taps, generator=g, dtype=torch.float64)
        ref = x + F.conv1d(F.pad(x.t()[None], (taps - 1, 0)), u[:, None, :], groups=48)[0].t()
        assert torch.allclose(B.input_convolution(x, u), ref, atol=1e-12)


def test_plain_rotation_is_a_rotation():
    g = torch.Generator().manual_seed(2)
    v = torch.randn(5, 3, 10, generator=g, dtype=torch.float64)
    pos = torch.tensor([0, 1, 5, 41, 1000])
    freq = B.frequencies(100.0, 6, None)
    out = B.rotate_half_split(v, pos, freq)
    assert torch.equal(out[..., 6:], v[..., 6:]) and torch.allclose(out[0], v[0])
    for i in range(3):
        a = pos.double() * freq[i]
        z = torch.complex(v[..., i], v[..., i + 3]) * torch.polar(torch.ones_like(a), a)[:, None]
        assert torch.allclose(out[..., i], z.real, atol=1e-12) and torch.allclose(out[..., i + 3], z.imag, atol=1e-12)


def test_plain_softmax_with_one_more_entry_and_the_soft_cap():
    g = torch.Generator().manual_seed(3)
    s = torch.randn(4, 7, generator=g, dtype=torch.float64) * 3
    s[1, 3:] = -math.inf
    ref = torch.softmax(torch.cat([s, torch.zeros(4, 1, dtype=torch.float64)], dim=1), dim=1)[:, :-1]   # (an entry of score 0)
    assert torch.allclose(B.softmax_with_one(s), ref, atol=1e-12)
    assert torch.allclose(B.softmax_with_one(s - 900.0), torch.zeros_like(s))          # far below the added 1
    x = torch.tensor([-1e4, -1.0, 0.0, 0.01, 1e4], dtype=torch.float64)
    y = B.soft_cap(x, 7.0)
    assert abs(float(y[0]) + 7.0) < 1e-9 and abs(float(y[4]) - 7.0) < 1e-9 and float(y[2]) == 0 and abs(float(y[3]) - 0.01) < 1e-6


def test_plain_recurrence_of_two_tokens_by_hand_and_its_limits():
    g = torch.Generator().manual_seed(4)
    W, H, d, dv = 10, 2, 3, 4
    r = lambda *s: torch.randn(*s, generator=g, dtype=torch.float64)
    w = {"q": r(H * d, W), "f": r(H * d, W), "f.b": r(H * d), "lower": torch.rand(H * d, generator=g, dtype=torch.float64),
         "v": r(H * dv, W), "norm": r(dv), "o": torch.eye(H * dv, dtype=torch.float64)}
    m = {"heads": H, "dim": d, "vdim": dv}
    h = r(2, W)
    y, S = B.hgrn2(h, w, "", m, 1e-6)
    for hh in range(H):
        rows, vals = slice(hh * d, hh * d + d), slice(hh * dv, hh * dv + dv)
        f = [w["lower"][rows] + (1 - w["lower"][rows]) * torch.sigmoid((w["f"] @ h[t] + w["f.b"])[rows]) for t in range(2)]
        v = [(w["v"] @ h[t])[vals] for t in range(2)]
        q = F.silu((w["q"] @ h[1])[rows])
        s1 = torch.outer(1 - f[0], v[0])
        s2 = f[1][:, None] * s1 + torch.outer(1 - f[1], v[1])
        assert torch.allclose(S[hh], s2)
        assert torch.allclose(y[1, vals], F.rms_norm(s2.t() @ q, (dv,), w["norm"], 1e-6))
    # a gate that never forgets writes nothing; one that always forgets (and may) writes the value itself
    w["f.b"] = torch.full((H * d,), 1e3, dtype=torch.float64)
    assert float(B.hgrn2(h, w, "", m, 1e-6)[1].abs().max()) == 0
    w["f.b"], w["lower"] = -w["f.b"], torch.zeros(H * d, dtype=torch.float64)
    assert torch.allclose(B.hgrn2(h, w, "", m, 1e-6)[1][0], (w["v"] @ h[1])[:dv].expand(d, dv))


def test_plain_mixture_weighs_what_an_expert_reads():
    z = torch.tensor([[0.1, 2.0, -1.0, 1.5, 0.3]], dtype=torch.float64)
    ids, wts = B.route_sigmoid(z, 2)
    assert ids.tolist() == [[1, 3]] and torch.allclose(wts, torch.sigmoid(torch.tensor([[2.0, 1.5]], dtype=torch.float64)))
    g = torch.Generator().manual_seed(5)
    r = lambda *s: torch.randn(*s, generator=g, dtype=torch.float64)
    w = {"router": torch.zeros(1, 6, dtype=torch.float64), "e0.gate": r(4, 6), "e0.up": r(4, 6), "e0.down": r(6, 4)}
    h = r(3, 6)
    half = F.silu(0.5 * h @ w["e0.gate"].T) * (0.5 * h @ w["e0.up"].T) @ w["e0.down"].T        # (a sigmoid of 0 is a half)
    assert torch.allclose(B.mixture(h, w, "", {"router": {"top": 1}}), half)
    assert not torch.allclose(half, 0.5 * B.expert(h, w, "e0."))


def test_plain_depth_average():
    rs = [torch.full((2, 3), float(10 ** j), dtype=torch.float64) for j in range(3)]
    out = B.depth_average(torch.tensor([2.0, -1.0, 0.5], dtype=torch.float64), rs)
    assert torch.equal(out, torch.full((2, 3), 2.0 - 10.0 + 50.0, dtype=torch.float64))
    assert config_from_dict(BD).to_model_spec().layers[3].depth_average.index == 3
