"""The Busadra decoder through the engine (model registry, loader, cache manager, step function, scheduler, entry
point) against the plain implementation, in every cutting of the requests."""
import copy
import json

import pytest
import torch

import qwen_engine_amd  # noqa: F401
from plain import busadra_plain as B
import traces
from busadra_tiny import BA, TINY, make_folder, random_config, random_tensors, write_folder

pytestmark = pytest.mark.gpu


@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    tmp = tmp_path_factory.mktemp("busadra")
    return {which: make_folder(tmp, which) for which in TINY}


def _requests(vocab, lengths, seed):
    g = torch.Generator().manual_seed(seed)
    return {f"q{i}": torch.randint(0, vocab, (n,), generator=g).tolist() for i, n in enumerate(lengths)}


def _reference(folder, reqs):
    cfg, w = B.read_folder(folder)
    return {rid: B.forward(cfg, w, toks).float() for rid, toks in reqs.items()}


def _tail_cut(reqs, tail=20):
    """All but the last ``tail`` tokens in one step (at least one), the rest one by one."""
    t = traces.Trace()
    for rid, toks in reqs.items():
        n = max(1, len(toks) - tail)
        t.step([(rid, toks[:n])], end=[rid] if n == len(toks) else [])
        for i in range(n, len(toks)):
            t.step([(rid, toks[i:i + 1])], end=[rid] if i == len(toks) - 1 else [])
    return t


CUTS = {"whole": traces.whole, "tail": _tail_cut, "portions": traces.portions, "mixed": lambda r: traces.mixed(r, seed=3)}


def _position_errors(got, ref):
    out = []
    for rid, rows in ref.items():
        scale = float(rows.abs().max())
        out += [float((torch.from_numpy(got[rid][p]) - rows[p]).abs().max()) / scale for p in range(rows.shape[0])]
    return torch.tensor(out)


def _every_expert(cfg):
    """The configuration with every expert chosen: in bfloat16 a router's close call may fall the other way, and the
    recurrences and convolutions carry such a choice on to later positions; without choices only rounding is left."""
    cfg = copy.deepcopy(cfg)
    for layer in cfg["layers"]:
        if layer["mlp"]:
            layer["mlp"]["router"]["top"] = layer["mlp"]["router"]["experts"]
    return cfg


def _assert_close(got, ref, what, choices=False):
    """bfloat16 against 64-bit: every position agrees to rounding; with ``choices`` (routers that pick) the typical one."""
    err = _position_errors(got, ref)
    assert not torch.isnan(err).any(), what
    assert float(err.median()) < 1.5e-2, f"{what}: median error {float(err.median())}"
    if not choices:
        assert float(err.quantile(0.95)) < 2.5e-2 and float(err.max()) < 7e-2, f"{what}: {float(err.max())}"


@pytest.mark.parametrize("cut", sorted(CUTS))
@pytest.mark.parametrize("which", sorted(TINY))
def test_every_cutting_in_float32(folders, tmp_path, which, cut):
    """Prompts longer than every window of the tiny models (so that pages go back while a request runs), of one
    and of two tokens, in every cutting, with poisoned pages."""
    cfg, _, page = TINY[which]
    reqs = _requests(cfg["vocab"], (70, 33, 121, 58, 2, 95, 1), seed=7)
    ref = _reference(folders[which], reqs)
    trace = CUTS[cut](reqs)
    out = str(tmp_path / "out")
    traces.run_in_process(trace, folders[which], "float32", out, page)
    got = traces.collect(trace, out, cfg["vocab"])
    bad, worst = traces.first_mismatch(got, ref, 2e-4)
    assert bad is None, f"first wrong logits at (request, position, relative error) {bad}"


@pytest.mark.parametrize("choices", [False, True])
@pytest.mark.parametrize("which", sorted(TINY))
def test_bfloat16_agrees_with_the_plain_model_and_with_itself_in_every_cutting(tmp_path, which, choices):
    cfg, seed, page = TINY[which]
    page = 16 if which in "AB" else page      # (pages of 16: the matrix-unit kernels where the sizes allow them)
    cfg = cfg if choices else _every_expert(cfg)
    folder = write_folder(str(tmp_path / "model"), cfg, random_tensors(cfg, seed))
    reqs = _requests(cfg["vocab"], (70, 33, 121, 58), seed=8)
    ref = _reference(folder, reqs)
    got = {}
    for cut in ("whole", "mixed", "portions"):
        trace = CUTS[cut](reqs)
        out = str(tmp_path / cut)
        traces.run_in_process(trace, folder, "bfloat16", out, page)
        got[cut] = traces.collect(trace, out, cfg["vocab"])
        _assert_close(got[cut], ref, f"{cut} against the plain model", choices)
    whole = {rid: torch.stack([torch.from_numpy(got["whole"][rid][p]) for p in range(len(t))]) for rid, t in reqs.items()}
    for cut in ("mixed", "portions"):
        _assert_close(got[cut], whole, f"{cut} against whole prompts", choices)


def test_long_decoding_over_many_pages_and_windows(folders, tmp_path):
    cfg, _, page = TINY["A"]
    reqs = _requests(cfg["vocab"], (340,), seed=9)
    ref = _reference(folders["A"], reqs)
    trace = traces.tail_decoded(reqs, tail=335)               # five tokens of prompt, then one at a time
    out = str(tmp_path / "out")
    traces.run_in_process(trace, folders["A"], "float32", out, page)
    bad, worst = traces.first_mismatch(traces.collect(trace, out, cfg["vocab"]), ref, 2e-4)
    assert bad is None, f"first wrong logits at (request, position, relative error) {bad}"


def _one_layer(kind, tmp_path, name, sharpen, mixer=None, taps=3):
    """A model of one layer of BA (by its type), with the named tensors changed by the functions given."""
    layer = copy.deepcopy(next(l for l in BA["layers"] if l["type"] == kind and l["mlp"] is not None))
    layer["mixer"].update(mixer or {})
    cfg = dict(BA, layers=[layer], canon={"taps": taps})
    w = random_tensors(cfg, 31, torch.float32)
    for n, f in sharpen.items():
        w[n] = f(w[n])
    return cfg, write_folder(str(tmp_path / name), cfg, w)


def test_a_far_token_decides_the_logits_through_the_state(tmp_path):
    """One recurrent layer whose gates (almost) never forget: the logits at the end depend on the identity of one early
    token hundreds of positions back, by as much in the engine as in the plain model."""
    cfg, folder = _one_layer("hgrn2", tmp_path, "model", {"l0.mix.lower": lambda t: torch.full_like(t, 0.999)})
    g = torch.Generator().manual_seed(10)
    base = torch.randint(0, cfg["vocab"], (400,), generator=g).tolist()
    other = list(base)
    other[3] = (base[3] + 1) % cfg["vocab"]
    cfg_, w_ = B.read_folder(folder)
    reqs = {"a": base, "b": other}
    ref = {rid: B.forward(cfg_, w_, t).float() for rid, t in reqs.items()}
    delta = float((ref["a"][-1] - ref["b"][-1]).abs().max())
    assert delta > 2e-3 * float(ref["a"].abs().max())
    for name, trace in (("tail", traces.tail_decoded(reqs, tail=40)), ("portions", traces.portions(reqs))):
        out = str(tmp_path / name)
        traces.run_in_process(trace, folder, "float32", out, 8)
        got = traces.collect(trace, out, cfg["vocab"])
        bad, worst = traces.first_mismatch(got, ref, 1e-4)
        assert bad is None, f"{name}: first wrong logits at (request, position, relative error) {bad}"
        assert abs(float((torch.from_numpy(got["a"][399] - got["b"][399])).abs().max()) - delta) < 0.05 * delta


@pytest.mark.parametrize("window,taps", [(37, 1), (16, 1), (3, 1), (12, 3), (20, 6)])
def test_a_token_at_the_windows_edge_decides_and_one_behind_it_does_not(tmp_path, window, taps):
    """One windowed layer.  Changing the token at position p changes the keys of p and of the taps - 1 positions whose
    convolution reads it, the outputs of the queries that see one of those, and what the second convolution makes of
    them: the last position that can tell is p + window - 1 + 2 (taps - 1).  It does, and the logits of the next stay
    exactly as they were, in prompts' portions and in decoding, in the engine as in the plain model."""
    cfg, folder = _one_layer("attention", tmp_path, "model", {"l0.mix.q": lambda t: 2.0 * t}, mixer={"mask": {"size": window}}, taps=taps)
    g = torch.Generator().manual_seed(11)
    base = torch.randint(0, cfg["vocab"], (130,), generator=g).tolist()
    p = 40
    other = list(base)
    other[p] = (base[p] + 1) % cfg["vocab"]
    cfg_, w_ = B.read_folder(folder)
    ref = {"a": B.forward(cfg_, w_, base).float(), "b": B.forward(cfg_, w_, other).float()}
    last_in = p + window - 1 + 2 * (taps - 1)
    first_out = last_in + 1
    assert float((ref["a"][last_in] - ref["b"][last_in]).abs().max()) > 1e-5 * float(ref["a"].abs().max())
    assert torch.equal(ref["a"][first_out:], ref["b"][first_out:])
    reqs = {"a": base, "b": other}
    for name, trace in (("portions", traces.portions(reqs)), ("decoded", traces.tail_decoded(reqs, tail=130 - p - 2))):
        out = str(tmp_path / name)
        traces.run_in_process(trace, folder, "float32", out, 8)
        got = traces.collect(trace, out, cfg["vocab"])
        bad, worst = traces.first_mismatch(got, ref, 1e-4)
        assert bad is None, f"{name}: first wrong logits at (request, position, relative error) {bad}"
        assert not (got["a"][last_in] == got["b"][last_in]).all()
        for q in range(first_out, 130):
            assert (got["a"][q] == got["b"][q]).all(), f"{name}: position {q} still sees position {p}"


def test_slots_and_pages_that_come_back_start_clean(folders):
    """A request that takes over the pages of one that ended computes what it computes alone."""
    from qwen_engine_amd.engine import ModelRunner, StepEntry, load_model
    cfg, _, page = TINY["A"]
    reqs = _requests(cfg["vocab"], (40, 37), seed=11)
    ref = _reference(folders["A"], reqs)
    runner = ModelRunner(load_model(folders["A"], dtype="float32"), page_size=page, num_pages=6, max_requests=1,
                         debug_poison=True)
    for rid in ("q0", "q1", "q0"):
        toks = reqs[rid]
        runner.add_request(rid)
        a = runner.step([StepEntry(rid, toks[:5], [4])])
        b = runner.step([StepEntry(rid, toks[5:], list(range(len(toks) - 5)))])
        runner.free_request(rid)
        runner.cache.check_invariants()
        got = torch.cat([a, b]).cpu()
        err = float((got - ref[rid][4:]).abs().max()) / float(ref[rid].abs().max())
        assert err < 2e-4, f"{rid}: {err}"


def test_windows_give_their_pages_back_while_the_request_runs(folders):
    """Model A's two attention layers have windows of 37 and 9 keys; a request of 200 tokens never holds more pages of
    a group than its window spans."""
    from qwen_engine_amd.engine import ModelRunner, StepEntry, load_model
    cfg, _, page = TINY["A"]
    toks = _requests(cfg["vocab"], (200,), seed=12)["q0"]
    runner = ModelRunner(load_model(folders["A"], dtype="float32"), page_size=page, num_pages=40, max_requests=1)
    runner.add_request("r")
    assert [gs.window for gs in runner.cache.groups] == [37, 9]
    most = [0, 0]
    for i in range(0, 200, 10):
        runner.step([StepEntry("r", toks[i:i + 10], [])])
        for grp in range(2):
            most[grp] = max(most[grp], sum(1 for pg in runner.cache.requests["r"].tables[grp] if pg >= 0))
    assert most[0] <= (37 + 10) // page + 2 and most[1] <= (9 + 10) // page + 2
    runner.free_request("r")
    runner.cache.check_invariants()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_greedy_generation_through_the_entry_point(folders, dtype):
    from qwen_engine_amd import EngineConfig, SamplingParams, generate
    cfg, _, page = TINY["B"]
    cfg_, w_ = B.read_folder(folders["B"])
    prompts = list(_requests(cfg["vocab"], (19, 3, 44), seed=12).values())
    res = generate(folders["B"], prompts, SamplingParams(max_new_tokens=12, ignore_eos=True),
                   EngineConfig(dtype=dtype, block_size=page, max_num_seqs=2, max_model_len=64, max_step_tokens=32,
                                prefill_chunk=8, debug_poison=True))
    off = 0
    for prompt, r in zip(prompts, res):
        assert r.finish_reason == "length" and len(r.token_ids) == 12
        logits = B.forward(cfg_, w_, prompt + r.token_ids[:-1]).float()
        for i, tok in enumerate(r.token_ids):
            row = logits[len(prompt) - 1 + i]
            if dtype == "float32":
                assert tok == int(row.argmax()), f"token {i} of a prompt of {len(prompt)}"
            else:
                off += not float(row.max() - row[tok]) <= 3e-2 * float(row.abs().max())
    # (in bfloat16 a router that picks one expert of four may pick another on a close call: few tokens may differ)
    assert off <= 3, f"{off} of 36 tokens are not the plain model's choice for the engine's own sequence"


def test_recorded_decode_steps_give_the_logits_of_steps_run_as_they_come(folders):
    """The same tokens through a runner that records its steps and one that runs them as they come.  (A recorded prompt
    portion is filled up to a round length, so its products run on other kernels and round otherwise: the logits agree
    to rounding but for a router's close calls, not bit for bit.)"""
    from qwen_engine_amd.engine import ModelRunner, StepEntry, load_model
    cfg, _, page = TINY["B"]
    model = load_model(folders["B"], dtype="bfloat16")
    prompts = list(_requests(cfg["vocab"], (21, 9, 30), seed=13).values())
    fed, outs = [], []
    for use_graphs in (False, True):
        runner = ModelRunner(model, page_size=page, num_pages=24, max_requests=3, use_graphs=use_graphs)
        rows = []
        for i, p in enumerate(prompts):
            runner.add_request(i)
            rows.append(runner.step([StepEntry(i, p, [len(p) - 1])]).cpu())
        steps = [torch.cat(rows)]
        for k in range(10):
            if not use_graphs:
                fed.append([int(r.argmax()) for r in steps[-1]])
            steps.append(runner.step([StepEntry(i, [fed[k][i]], [0]) for i in range(3)]).cpu())
        outs.append(torch.cat(steps))
        if use_graphs:
            assert runner.graph_steps_of["decode"] == 10
    assert not torch.isnan(outs[1]).any()
    err = (outs[0] - outs[1]).abs().amax(dim=1) / float(outs[0].abs().max())
    assert float(err.median()) < 1.5e-2 and float((err > 6e-2).float().mean()) <= 0.1, err


def test_middling_sizes_on_the_matrix_unit_kernels(tmp_path):
    """Sizes at which the bfloat16 mode runs the matrix-unit kernels inside the engine (paged attention under a window with
    a soft cap, chunked recurrences over several chunks, the tiled grouped product of the experts): prompts of hundreds of
    tokens, whole and in a mixed schedule, in both element types."""
    moe = lambda ff, e, top: {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": e, "top": top}}
    cfg = {
        "architecture": "Busadra", "vocab": 400, "width": 256, "norm": {"eps": 1e-5}, "canon": {"taps": 4}, "logit_scale": 0.5,
        "layers": [
            {"type": "hgrn2", "mixer": {"heads": 6, "dim": 32, "vdim": 80}, "mlp": moe(64, 12, 4)},
            {"type": "attention",
             "mixer": {"heads": 8, "kv_heads": 2, "dim": 64, "vdim": 128, "mask": {"size": 150}, "scale": 0.15, "softcap": 6.0,
                       "rot": {"base": 10000.0, "dims": 32, "scaling": {"factor": 4.0, "low": 1.0, "high": 4.0, "original": 256}}},
             "mlp": moe(96, 5, 3)},
            {"type": "hgrn2", "mixer": {"heads": 3, "dim": 104, "vdim": 128}, "mlp": moe(128, 6, 2)},
            {"type": "attention",
             "mixer": {"heads": 6, "kv_heads": 6, "dim": 128, "vdim": 64, "mask": {"size": 100}, "scale": 0.1, "softcap": 20.0,
                       "rot": {"base": 500.0, "dims": 128, "scaling": {"factor": 8.0, "low": 1.0, "high": 4.0, "original": 1000}}},
             "mlp": moe(64, 8, 2)},
        ],
    }
    reqs = _requests(cfg["vocab"], (420, 300, 37, 260), seed=14)
    for dtype in ("float32", "bfloat16"):
        c = cfg if dtype == "float32" else _every_expert(cfg)
        folder = write_folder(str(tmp_path / dtype), c, random_tensors(c, 41))
        ref = _reference(folder, reqs)
        for cut in ("whole", "mixed"):
            trace = CUTS[cut](reqs)
            out = str(tmp_path / f"{dtype}_{cut}")
            traces.run_in_process(trace, folder, dtype, out, 16)
            got = traces.collect(trace, out, cfg["vocab"])
            if dtype == "float32":
                bad, worst = traces.first_mismatch(got, ref, 3e-4)
                assert bad is None, f"{cut}: first wrong logits at (request, position, relative error) {bad}"
            else:
                _assert_close(got, ref, f"{dtype} {cut}")


def test_recorded_prompt_portions_give_the_logits_of_portions_run_as_they_come(folders):
    """Portions of a round length are recorded and replayed, for one request after another, between steps of other kinds."""
    from qwen_engine_amd.engine import ModelRunner, StepEntry, load_model
    cfg, _, page = TINY["B"]
    model = load_model(folders["B"], dtype="bfloat16")
    reqs = _requests(cfg["vocab"], (560, 530), seed=15)
    outs = []
    for use_graphs in (False, True):
        runner = ModelRunner(model, page_size=page, num_pages=80, max_requests=2, use_graphs=use_graphs)
        rows = []
        for rid, toks in reqs.items():
            runner.add_request(rid)
            rows.append(runner.step([StepEntry(rid, toks[:256], [255])]).cpu())
            rows.append(runner.step([StepEntry(rid, toks[256:512], [255])]).cpu())
            rows.append(runner.step([StepEntry(rid, toks[512:], [3])]).cpu())
        outs.append(torch.cat(rows))
        if use_graphs:
            assert runner.graph_steps_of["portion"] == 4
    assert torch.equal(outs[0], outs[1])


@pytest.mark.parametrize("seed", [3, 4, 5, 11, 24, 27])
def test_configurations_drawn_at_random(tmp_path, seed):
    """Layer orders, head counts, sizes, windows and constants that no other test names, in float32 against the plain
    model, whole and in a mixed schedule."""
    cfg = random_config(seed)
    folder = write_folder(str(tmp_path / "model"), cfg, random_tensors(cfg, seed))
    reqs = _requests(cfg["vocab"], (330, 37, 150, 2, 90), seed=seed)
    ref = _reference(folder, reqs)
    for cut in ("whole", "mixed"):
        trace = CUTS[cut](reqs)
        out = str(tmp_path / cut)
        traces.run_in_process(trace, folder, "float32", out, 16)
        bad, worst = traces.first_mismatch(traces.collect(trace, out, cfg["vocab"]), ref, 3e-4)
        assert bad is None, f"{cut}: first wrong logits at (request, position, relative error) {bad}"


def test_the_command_line_with_random_weights(tmp_path, capsys):
    """main.py writes random weights for a Busadra config.json and generates from token ids."""
    import main as cli
    cfg, _, page = TINY["C"]
    cfg_path = tmp_path / "config.json"
    cfg_path.write_text(json.dumps(cfg))
    folder = str(tmp_path / "model")
    rc = cli.main(["--model-name-or-path", folder, "--random-weights", str(cfg_path), "--seed", "3", "--prompt-ids", "5,17,3",
                   "--prompt-ids", "9,9,100,41", "--max-new-tokens", "6", "--block-size", "16", "--max-model-len", "64",
                   "--ignore-eos", "--stats"])
    assert rc == 0
    out = capsys.readouterr().out
    assert out.count("Prompt:") == 2 and "5 17 3" in out
    stats = json.loads(out.strip().splitlines()[-1])
    assert stats["graph_steps_decode"] >= 4                 # single new tokens were replayed from recorded steps
    cfg_, w_ = B.read_folder(folder)
    assert set(w_) == set(random_tensors(cfg, 0))           # every tensor of the design, by its name


def test_the_replay_program_on_a_folder_with_tensors_around_a_missing_feed_forward(folders, tmp_path):
    """bin/trace_run as a user runs it, on a copy of model A whose layer without a feed-forward still has the tensors that
    would stand around one: they change nothing."""
    cfg, seed, page = TINY["A"]
    w = random_tensors(cfg, seed)
    width, taps = cfg["width"], cfg["canon"]["taps"]
    w.update({"l1.norm2": torch.randn(width).bfloat16(), "l1.canon2": torch.randn(width, taps).bfloat16(),
              "l1.ls2": torch.randn(width).bfloat16()})
    folder = write_folder(str(tmp_path / "model"), cfg, w)
    reqs = _requests(cfg["vocab"], (40, 9), seed=16)
    ref = _reference(folders["A"], reqs)
    trace = CUTS["mixed"](reqs)
    out = str(tmp_path / "out")
    traces.run_program(trace, folder, "float32", out, page)
    bad, worst = traces.first_mismatch(traces.collect(trace, out, cfg["vocab"]), ref, 2e-4)
    assert bad is None, f"first wrong logits at (request, position, relative error) {bad}"
