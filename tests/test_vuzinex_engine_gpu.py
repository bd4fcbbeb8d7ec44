"""The Vuzinex decoder through the engine (model registry, loader, cache manager, step function, scheduler, entry point)
against the plain implementation, in every cutting of the requests."""
import copy
import json

import pytest
import torch

import qwen_engine_amd  # noqa: F401
from plain import vuzinex_plain as B
import traces
from vuzinex_tiny import TINY, VA, make_folder, random_config, random_tensors, write_folder

pytestmark = pytest.mark.gpu


@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    tmp = tmp_path_factory.mktemp("vuzinex")
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


def _run(trace, folder, dtype, out, page, vocab):
    traces.run_in_process(trace, folder, dtype, str(out), page)
    return traces.collect(trace, str(out), vocab)


def _assert_close(got, ref, what):
    """bfloat16 against 64-bit: the typical position agrees to rounding, none is far off."""
    err = []
    for rid, rows in ref.items():
        scale = float(rows.abs().max())
        err += [float((torch.from_numpy(got[rid][p]) - rows[p]).abs().max()) / scale for p in range(rows.shape[0])]
    err = torch.tensor(err)
    assert not torch.isnan(err).any(), what
    assert float(err.median()) < 2.5e-2 and float(err.quantile(0.95)) < 6e-2 and float(err.max()) < 0.2, \
        f"{what}: median {float(err.median())}, 95% {float(err.quantile(0.95))}, max {float(err.max())}"


@pytest.mark.parametrize("cut", sorted(CUTS))
@pytest.mark.parametrize("which", sorted(TINY))
def test_every_cutting_in_float32(folders, tmp_path, which, cut):
    """Prompts longer than every chunk but one of the tiny models, of one and of two tokens, in every cutting, with
    poisoned pages."""
    cfg, _, page = TINY[which]
    reqs = _requests(cfg["vocab"], (70, 33, 121, 58, 2, 95, 1), seed=7)
    ref = _reference(folders[which], reqs)
    bad, worst = traces.first_mismatch(_run(CUTS[cut](reqs), folders[which], "float32", tmp_path / "out", page, cfg["vocab"]), ref, 3e-4)
    assert bad is None, f"first wrong logits at (request, position, relative error) {bad}"


@pytest.mark.parametrize("which", sorted(TINY))
def test_bfloat16_agrees_with_the_plain_model_and_with_itself_in_every_cutting(folders, tmp_path, which):
    cfg, _, page = TINY[which]
    page = 16 if which in "AB" else page      # (pages of 16: the matrix-unit kernels where the sizes allow them)
    reqs = _requests(cfg["vocab"], (70, 33, 121, 58), seed=8)
    ref = _reference(folders[which], reqs)
    got = {}
    for cut in ("whole", "mixed", "portions"):
        got[cut] = _run(CUTS[cut](reqs), folders[which], "bfloat16", tmp_path / cut, page, cfg["vocab"])
        _assert_close(got[cut], ref, f"{cut} against the plain model")
    whole = {rid: torch.stack([torch.from_numpy(got["whole"][rid][p]) for p in range(len(t))]) for rid, t in reqs.items()}
    for cut in ("mixed", "portions"):
        _assert_close(got[cut], whole, f"{cut} against whole prompts")


def test_long_decoding_over_many_pages_and_chunks(folders, tmp_path):
    cfg, _, page = TINY["A"]
    reqs = _requests(cfg["vocab"], (340,), seed=9)
    trace = traces.tail_decoded(reqs, tail=335)               # five tokens of prompt, then one at a time
    got = _run(trace, folders["A"], "float32", tmp_path / "out", page, cfg["vocab"])
    bad, worst = traces.first_mismatch(got, _reference(folders["A"], reqs), 3e-4)
    assert bad is None, f"first wrong logits at (request, position, relative error) {bad}"


def _one_layer(kind, tmp_path, name, change=None, mixer=None):
    """A model of one layer of VA (by its type) run once, with its mixer's entries and named tensors changed."""
    layer = copy.deepcopy(next(l for l in VA["layers"] if l["type"] == kind))
    for path, v in (mixer or {}).items():
        cur = layer["mixer"]
        for k in path.split(".")[:-1]:
            cur = cur[k]
        cur[path.split(".")[-1]] = v
    cfg = dict(VA, layers=[layer], loop=None)
    w = random_tensors(cfg, 31, torch.float32)
    for n, f in (change or {}).items():
        w[n] = f(w[n])
    return cfg, write_folder(str(tmp_path / name), cfg, w)


FAR = {
    # (a forget gate, decays or step sizes that (almost) never forget; the other mixer of the layer weighs little)
    "mlstm": ("parallel", {"l0.mix.right.f.b": lambda t: t + 50.0}, {"left_scale": 0.01, "right.gate_cap": 15.0}),
    "gla": ("parallel_2", {"l0.mix.right.a2.b": lambda t: t + 12.0}, {"left_scale": 0.01}),
    "mamba2": ("mamba2", {"l0.mix.A_log": lambda t: t - 9.0}, {}),
    # (one score that stands out: q and k of a head's unrotated numbers are large where the token is the one asked for)
    "attention": ("parallel_2", {"l0.mix.left.q.norm": lambda t: 3.0 * t}, {"right_scale": 0.01}),
}


@pytest.mark.parametrize("which", sorted(FAR))
def test_a_far_token_decides_the_logits(tmp_path, which):
    """The logits at the end depend on the identity of one early token hundreds of positions back, through a state or an
    old key, by as much in the engine as in the plain model."""
    kind, change, mixer = FAR[which]
    cfg, folder = _one_layer(kind, tmp_path, "model", change, mixer)
    g = torch.Generator().manual_seed(10)
    base = torch.randint(0, cfg["vocab"], (400,), generator=g).tolist()
    other = list(base)
    other[3] = (base[3] + 1) % cfg["vocab"]
    reqs = {"a": base, "b": other}
    ref = _reference(folder, reqs)
    delta = float((ref["a"][-1] - ref["b"][-1]).abs().max())
    assert delta > 5e-4 * float(ref["a"].abs().max())
    for name, trace in (("tail", traces.tail_decoded(reqs, tail=40)), ("portions", traces.portions(reqs))):
        got = _run(trace, folder, "float32", tmp_path / name, 8, cfg["vocab"])
        bad, worst = traces.first_mismatch(got, ref, 1.5e-4)
        assert bad is None, f"{name}: first wrong logits at (request, position, relative error) {bad}"
        assert abs(float((torch.from_numpy(got["a"][399] - got["b"][399])).abs().max()) - delta) < 0.1 * delta


@pytest.mark.parametrize("chunk", [37, 16, 1, 8])
def test_a_token_is_seen_to_the_end_of_its_chunk_and_not_beyond(tmp_path, chunk):
    """One layer of chunked attention whose other mixer carries nothing.  The token at position p changes its own key
    and, through the embedding of pairs, that of p + 1; the last position that can tell is the end of p + 1's chunk.
    It does, and the logits of the next stay exactly as they were, in prompts' portions and in decoding."""
    cfg, folder = _one_layer("parallel", tmp_path, "model", {"l0.mix.left.q": lambda t: 2.0 * t, "l0.mix.left.sink": lambda t: t - 3.0},
                             {"left.mask.size": chunk, "right_scale": 0.0})
    g = torch.Generator().manual_seed(11)
    base = torch.randint(0, cfg["vocab"], (130,), generator=g).tolist()
    p = 40
    other = list(base)
    other[p] = (base[p] + 1) % cfg["vocab"]
    reqs = {"a": base, "b": other}
    ref = _reference(folder, reqs)
    first_out = ((p + 1) // chunk + 1) * chunk
    last_in = first_out - 1
    assert float((ref["a"][last_in] - ref["b"][last_in]).abs().max()) > 1e-4 * float(ref["a"].abs().max())
    assert torch.equal(ref["a"][first_out:], ref["b"][first_out:])
    for name, trace in (("portions", traces.portions(reqs)), ("decoded", traces.tail_decoded(reqs, tail=130 - p - 2))):
        got = _run(trace, folder, "float32", tmp_path / name, 8, cfg["vocab"])
        bad, worst = traces.first_mismatch(got, ref, 1e-4)
        assert bad is None, f"{name}: first wrong logits at (request, position, relative error) {bad}"
        assert not (got["a"][last_in] == got["b"][last_in]).all()
        for q in range(first_out, 130):
            assert (got["a"][q] == got["b"][q]).all(), f"{name}: position {q} still sees position {p}"


def test_a_sink_takes_its_part_of_the_softmax(tmp_path):
    """Sinks far above every score leave nothing of the attention, sinks far below all of it: the two models differ by
    as much in the engine as in the plain model, at a first token and later."""
    toks = _requests(VA["vocab"], (60,), seed=3)["q0"]
    refs, gots = [], []
    for name, shift in (("high", 40.0), ("low", -40.0)):
        cfg, folder = _one_layer("parallel", tmp_path, name, {"l0.mix.left.sink": lambda t: t + shift})
        refs.append(_reference(folder, {"r": toks})["r"])
        got = _run(traces.portions({"r": toks}), folder, "float32", tmp_path / (name + "_out"), 8, cfg["vocab"])
        bad, _ = traces.first_mismatch(got, {"r": refs[-1]}, 1e-4)
        assert bad is None, bad
        gots.append(got["r"])
    for p in (0, 5, 59):
        d = float((refs[0][p] - refs[1][p]).abs().max())
        assert d > 1e-2 and abs(float(torch.from_numpy(gots[0][p] - gots[1][p]).abs().max()) - d) < 0.01 * d


def test_the_token_before_a_portion_chooses_the_row_of_pairs(tmp_path):
    """A model whose layer adds (almost) nothing: the logits are the embedding's, and change with the token before."""
    cfg, folder = _one_layer("mamba2", tmp_path, "model", {"l0.norm1b": lambda t: torch.full_like(t, -1.0)})
    toks = _requests(cfg["vocab"], (24,), seed=5)["q0"]
    ref = _reference(folder, {"r": toks})
    alone = _reference(folder, {"r": toks[10:11]})["r"][0]
    assert float((alone - ref["r"][10]).abs().max()) > 0.1 * float(alone.abs().max())     # (the first token's row is another)
    t = traces.Trace()
    for a, b in ((0, 1), (1, 2), (2, 4), (4, 10), (10, 11), (11, 13), (13, 24)):
        t.step([("r", toks[a:b])], end=["r"] if b == 24 else [])
    for dtype, tol in (("float32", 1e-5), ("bfloat16", 2e-2)):
        bad, _ = traces.first_mismatch(_run(t, folder, dtype, tmp_path / dtype, 8, cfg["vocab"]), ref, tol)
        assert bad is None, bad


def test_every_pass_of_a_loop_has_a_cache_and_a_state_of_its_own(folders, tmp_path):
    """Model A's layers 1 and 2 written out twice (other names, the same weights) give the logits of the loop."""
    cfg, seed, page = TINY["A"]
    w = random_tensors(cfg, seed)
    flat = copy.deepcopy(dict(cfg, loop=None))
    order = [0, 1, 2, 1, 2, 3]
    flat["layers"] = [copy.deepcopy(cfg["layers"][i]) for i in order]
    fw = {k: v for k, v in w.items() if not k.startswith("l")}
    for j, i in enumerate(order):
        fw.update({f"l{j}." + k.split(".", 1)[1]: v.clone() for k, v in w.items() if k.startswith(f"l{i}.")})
    folder = write_folder(str(tmp_path / "flat"), flat, fw)
    reqs = _requests(cfg["vocab"], (60, 45), seed=4)
    a = _run(CUTS["mixed"](reqs), folders["A"], "float32", tmp_path / "a", page, cfg["vocab"])
    b = _run(CUTS["mixed"](reqs), folder, "float32", tmp_path / "b", page, cfg["vocab"])
    assert all((a[r][p] == b[r][p]).all() for r in a for p in a[r])


def test_slots_and_pages_that_come_back_start_clean(folders):
    """A request that takes over the pages and the state slot of one that ended computes what it computes alone."""
    from qwen_engine_amd.engine import ModelRunner, StepEntry, load_model
    for which in "AD":
        cfg, _, page = TINY[which]
        reqs = _requests(cfg["vocab"], (40, 37), seed=11)
        ref = _reference(folders[which], reqs)
        runner = ModelRunner(load_model(folders[which], dtype="float32"), page_size=page, num_pages=-(-40 // page), max_requests=1,
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
            assert err < 3e-4, f"{which} {rid}: {err}"


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_greedy_generation_through_the_entry_point(folders, dtype):
    from qwen_engine_amd import EngineConfig, SamplingParams, generate
    cfg, _, page = TINY["B"]
    cfg_, w_ = B.read_folder(folders["B"])
    prompts = list(_requests(cfg["vocab"], (19, 3, 44), seed=12).values())
    res = generate(folders["B"], prompts, SamplingParams(max_new_tokens=12, ignore_eos=True),
                   EngineConfig(dtype=dtype, block_size=page, max_num_seqs=2, max_model_len=64, max_step_tokens=32,
                                prefill_chunk=8, debug_poison=True))
    for prompt, r in zip(prompts, res):
        assert r.finish_reason == "length" and len(r.token_ids) == 12
        logits = B.forward(cfg_, w_, prompt + r.token_ids[:-1]).float()
        for i, tok in enumerate(r.token_ids):
            row = logits[len(prompt) - 1 + i]
            if dtype == "float32":
                assert tok == int(row.argmax()), f"token {i} of a prompt of {len(prompt)}"
            else:
                assert float(row.max() - row[tok]) <= 5e-2 * float(row.abs().max()), f"token {i} of a prompt of {len(prompt)}"


def test_recorded_decode_steps_give_the_logits_of_steps_run_as_they_come(folders):
    """The same tokens through a runner that records its steps and one that runs them as they come; three requests, so that
    a recorded step for four rows (when a fourth came and went) is filled up too."""
    from qwen_engine_amd.engine import ModelRunner, StepEntry, load_model
    cfg, _, page = TINY["B"]
    model = load_model(folders["B"], dtype="bfloat16")
    prompts = list(_requests(cfg["vocab"], [21 + 3 * i for i in range(9)], seed=13).values())
    fed, outs = [], []
    for use_graphs in (False, True):
        runner = ModelRunner(model, page_size=page, num_pages=60, max_requests=9, use_graphs=use_graphs)
        rows = []
        for i, p in enumerate(prompts):
            runner.add_request(i)
            rows.append(runner.step([StepEntry(i, p, [len(p) - 1])]).cpu())
        steps = [torch.cat(rows)]
        for k in range(10):                                # (nine rows: recorded for sixteen, filled up)
            if not use_graphs:
                fed.append([int(r.argmax()) for r in steps[-1]])
            steps.append(runner.step([StepEntry(i, [fed[k][i]], [0]) for i in range(9)]).cpu())
        outs.append(torch.cat(steps))
        if use_graphs:
            assert runner.graph_steps_of["decode"] == 10
    assert not torch.isnan(outs[1]).any()
    err = (outs[0] - outs[1]).abs().amax(dim=1) / float(outs[0].abs().max())
    assert float(err.max()) < 3e-2, err


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


def test_middling_sizes_on_the_matrix_unit_kernels(tmp_path):
    """Sizes at which the bfloat16 mode runs the matrix-unit kernels inside the engine (paged attention in chunks and over
    all keys, chunked recurrences over several chunks, tiled products cut along K for the 32-bit columns): prompts of
    hundreds of tokens, whole and in a mixed schedule, in both element types."""
    cfg = {
        "architecture": "Vuzinex", "vocab": 400, "width": 512, "norm": {"eps": 1e-5}, "residual_mult": 0.8, "logit_scale": 0.6,
        "embedding": {"scale": 2.0, "bigram": {"buckets": 211, "mul_prev": 23, "mul_cur": 41}}, "loop": {"start": 1, "stop": 2, "times": 2},
        "layers": [
            {"type": "parallel_2", "mlp": {"kind": "dense", "ff": 320}, "mixer": {
                "left": {"heads": 8, "kv_heads": 2, "dim": 64, "vdim": 128, "scale": 0.15,
                         "rot": {"base": 10000.0, "dims": 32, "scaling": {"factor": 4.0, "original": 256, "fast": 16.0, "slow": 1.0}}},
                "right": {"heads": 6, "dim": 32, "vdim": 80, "tau": 8.0, "decay_rank": 12}, "left_scale": 1.1, "right_scale": 0.6}},
            {"type": "mamba2", "mlp": None, "mixer": {"heads": 8, "vdim": 64, "state": 96, "groups": 2, "conv": 4, "norm_groups": 2}},
            {"type": "parallel", "mlp": {"kind": "dense", "ff": 256}, "mixer": {
                "left": {"heads": 6, "kv_heads": 6, "dim": 128, "vdim": 64, "scale": 0.1, "mask": {"size": 100},
                         "rot": {"base": 500.0, "dims": 128, "scaling": {"factor": 8.0, "low": 1.0, "high": 4.0, "original": 1000}}},
                "right": {"heads": 3, "dim": 104, "vdim": 128, "gate_cap": 10.0}, "left_scale": 1.0, "right_scale": 0.9}},
        ],
    }
    reqs = _requests(cfg["vocab"], (420, 300, 37, 260), seed=14)
    folder = write_folder(str(tmp_path / "model"), cfg, random_tensors(cfg, 41))
    ref = _reference(folder, reqs)
    for dtype in ("float32", "bfloat16"):
        for cut in ("whole", "mixed"):
            got = _run(CUTS[cut](reqs), folder, dtype, tmp_path / f"{dtype}_{cut}", 16, cfg["vocab"])
            if dtype == "float32":
                bad, worst = traces.first_mismatch(got, ref, 4e-4)
                assert bad is None, f"{cut}: first wrong logits at (request, position, relative error) {bad}"
            else:
                _assert_close(got, ref, f"{dtype} {cut}")


@pytest.mark.parametrize("seed", [3, 4, 5, 11, 24, 27, 33, 38])
def test_configurations_drawn_at_random(tmp_path, seed):
    """Layer orders, head counts, sizes, chunks, loops and constants that no other test names, in float32 against the plain
    model, whole and in a mixed schedule."""
    cfg = random_config(seed)
    folder = write_folder(str(tmp_path / "model"), cfg, random_tensors(cfg, seed))
    reqs = _requests(cfg["vocab"], (230, 37, 110, 2, 90), seed=seed)
    ref = _reference(folder, reqs)
    for cut in ("whole", "mixed"):
        bad, worst = traces.first_mismatch(_run(CUTS[cut](reqs), folder, "float32", tmp_path / cut, 16, cfg["vocab"]), ref, 5e-4)
        assert bad is None, f"{cut}: first wrong logits at (request, position, relative error) {bad}"


def test_the_command_line_with_random_weights(tmp_path, capsys):
    """main.py writes random weights for a Vuzinex config.json and generates from token ids."""
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


def test_the_replay_program(folders, tmp_path):
    """bin/trace_run as a user runs it."""
    cfg, _, page = TINY["A"]
    reqs = _requests(cfg["vocab"], (40, 9), seed=16)
    trace = CUTS["mixed"](reqs)
    out = str(tmp_path / "out")
    traces.run_program(trace, folders["A"], "float32", out, page)
    bad, worst = traces.first_mismatch(traces.collect(trace, out, cfg["vocab"]), _reference(folders["A"], reqs), 3e-4)
    assert bad is None, f"first wrong logits at (request, position, relative error) {bad}"
