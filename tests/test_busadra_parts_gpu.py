"""Each mechanism of the Busadra layers alone: the kernel against the plain implementation's function of the same
mechanism (or a few lines of 64-bit torch), in float32 and bfloat16."""
import math

import pytest
import torch

import qwen_engine_amd  # noqa: F401
from plain import busadra_plain as B

pytestmark = pytest.mark.gpu
DEV = "cuda:0"


def ops():
    from qwen_engine_amd.kernels import ops as o
    return o


def rel(got, want):
    return float((got.double().cpu() - want.double()).abs().max()) / max(float(want.abs().max()), 1e-30)


def i32(v):
    return torch.tensor(v, dtype=torch.int32, device=DEV)


# Requests' rows fed in steps: portions beside single rows, portions of one and two rows, requests left out, single rows
# alone, a long portion
STEPS = [[(0, 5), (1, 1), (2, 2)], [(1, 1), (0, 1)], [(2, 1)], [(2, 37), (0, 2), (1, 5)], [(0, 150)], [(0, 1), (2, 1)],
         [(0, 17), (2, 70)]]
LENGTHS = {0: 176, 1: 7, 2: 111}
SLOT = {0: 2, 1: 0, 2: 3}


def _walk(call, inputs):
    """Feeds every request's rows through ``call(rows, table rows, portions, single)`` in STEPS; each request's outputs in
    order."""
    done = {s: 0 for s in LENGTHS}
    got = {s: [] for s in LENGTHS}
    for step in STEPS:
        rows, seq, at = [[] for _ in inputs], [], 0
        portions = []
        for s, n in step:
            for i, t in enumerate(inputs):
                rows[i].append(t[s][done[s]:done[s] + n])
            seq += [SLOT[s]] * n
            portions.append((at, n))
            at += n
        out = call([torch.cat(r).to(DEV) for r in rows], i32(seq), portions, all(n == 1 for _, n in step))
        at = 0
        for s, n in step:
            got[s].append(out[at:at + n].cpu())
            at += n
            done[s] += n
    assert done == LENGTHS
    return {s: torch.cat(v) for s, v in got.items()}


# ---- between two sublayers: scaled branch, average over depth, norm --------------------------------------------------
@pytest.mark.parametrize("T,H,parts,k", [(1, 96, 3, 5), (5, 202, 1, 0), (33, 2048, 4, 11), (700, 256, 2, 3), (3, 4096, 9, 20),
                                         (600, 1030, 1, 2), (2, 8200, 2, 4), (9, 70, 1, 9), (530, 8192, 1, 1), (4, 64, 0, 3)])
@pytest.mark.parametrize("center", [True, False])
def test_sums_average_and_norm(T, H, parts, k, center):
    g = torch.Generator().manual_seed(T + H)
    r = lambda *s: torch.randn(*s, generator=g)
    x, w, scale, coef = r(T, H) * 2.0 + 3.0, 1.0 + 0.3 * r(H), r(H), r(k + 1)
    delta = r(parts, T, H) if parts else None
    kept = r(k + 3, T, H)
    v = x.double() + (scale.double() * delta.double().sum(0) if parts else 0)
    want_x = B.depth_average(coef.double(), [kept[j].double() for j in range(k)] + [v])
    norm = B.layer_norm if center else B.rms_norm
    want = norm(want_x, w.double(), 1e-5)
    o = ops()
    args = dict(center=center, delta=None if delta is None else delta.to(DEV), scale=scale.to(DEV), index=k, coef=coef.to(DEV))
    xs, ks = x.to(DEV), kept.to(DEV)
    got = o.stream_norm(xs, w.to(DEV), 1e-5, torch.float32, kept=ks, **args)
    assert rel(got, want) < 6e-6 and rel(xs, want_x) < 2e-6
    assert rel(ks[k], v) < 1e-6                                     # this result kept, the others as they were
    assert torch.equal(ks[:k].cpu(), kept[:k]) and torch.equal(ks[k + 1:].cpu(), kept[k + 1:])
    # some rows only: nothing is written back
    rows = i32([T - 1, 0])
    xs, ks = x.to(DEV), kept.to(DEV)
    got = o.stream_norm(xs, w.to(DEV), 1e-5, torch.bfloat16, kept=ks, rows=rows, **args)
    assert rel(got, want[[T - 1, 0]]) < 6e-3 and torch.equal(xs.cpu(), x) and torch.equal(ks.cpu(), kept)
    # the sums alone; kept without an average; a branch in bfloat16
    o.stream_norm(xs, None, 0.0, torch.float32, kept=ks, **args)
    assert rel(xs, want_x) < 2e-6
    xs, ks = x.to(DEV), kept.to(DEV)
    b = r(T, H).bfloat16()
    got = o.stream_norm(xs, w.to(DEV), 1e-5, torch.bfloat16, center=center, delta=b.to(DEV), scale=scale.to(DEV), kept=ks, index=k)
    v = x.double() + scale.double() * b.double()
    assert rel(xs, v) < 1e-6 and torch.equal(ks[k].cpu(), xs.cpu()) and rel(got, norm(v, w.double(), 1e-5)) < 6e-3


@pytest.mark.parametrize("dtype,tol", [(torch.float32, 5e-6), (torch.bfloat16, 6e-3)])
@pytest.mark.parametrize("H,taps", [(96, 4), (70, 3), (256, 2), (202, 6), (64, 1), (2048, 4), (1030, 5), (4100, 4), (8200, 3)])
def test_norm_and_convolution_across_cuts_and_slots(dtype, tol, H, taps):
    """The convolution's input is the normed row, the earlier ones a request's state wherever it was cut; slots of other
    requests stay as they are."""
    g = torch.Generator().manual_seed(H + taps)
    x = {s: torch.randn(n, H, generator=g) * 2 + 1 for s, n in LENGTHS.items()}
    d = {s: torch.randn(n, H, generator=g) for s, n in LENGTHS.items()}
    w, u, sc = 1 + 0.3 * torch.randn(H, generator=g), torch.randn(H, taps, generator=g), torch.randn(H, generator=g)
    state = torch.full((4, taps - 1, H), float("nan"), device=DEV) if taps > 1 else None
    if taps > 1:
        for s in SLOT.values():
            state[s] = 0
    ut = u.t().contiguous().to(DEV)

    def call(rows, seq, portions, single):
        return ops().stream_norm(rows[0], w.to(DEV), 1e-5, dtype, center=True, delta=rows[1][None].contiguous(), scale=sc.to(DEV),
                                 conv_w=ut, state=state, tok_seq=seq, single_rows=single)

    got = _walk(call, [x, d])
    for s in LENGTHS:
        h = B.layer_norm(x[s].double() + sc.double() * d[s].double(), w.double(), 1e-5)
        assert rel(got[s], B.input_convolution(h, u.double())) < tol, s
        if taps > 1:
            last = torch.cat([torch.zeros(taps - 1, H, dtype=torch.float64), h])[-(taps - 1):]
            assert rel(state[SLOT[s]], last) < 5e-6
    if taps > 1:
        assert torch.isnan(state[1]).all()


# ---- the recurrence -----------------------------------------------------------------------------------------------------
def _plain_recurrence(q, z, v, low, H, D, Dv):
    f = low + (1 - low) * torch.sigmoid(z)
    write = (1 - low) * torch.sigmoid(-z)
    S = torch.zeros(H, D, Dv, dtype=torch.float64)
    out = []
    q = q * torch.sigmoid(q)
    for t in range(q.shape[0]):
        S = f[t].view(H, D, 1) * S + write[t].view(H, D, 1) * v[t].view(H, 1, Dv)
        out.append((S * q[t].view(H, D, 1)).sum(1))
    return torch.stack(out), S


@pytest.mark.parametrize("H,D,Dv", [(2, 12, 8), (3, 20, 36), (2, 64, 128), (1, 4, 200), (4, 128, 24), (5, 6, 7), (1, 200, 48), (2, 3, 5),
                                    (1, 256, 128), (3, 50, 130), (2, 90, 64), (16, 16, 16)])
@pytest.mark.parametrize("chunk", [0, 16, 64, 256])
def test_recurrence_with_a_forget_gate_across_cuts_and_slots(H, D, Dv, chunk):
    """Row by row, in chunks of several lengths, and (single new tokens) in one launch with the norm; gates from 0 to 1."""
    o = ops()
    g = torch.Generator().manual_seed(H * D + Dv)
    nk, nv = H * D, H * Dv
    y = {s: torch.randn(n, 2 * nk + nv, generator=g) * 1.5 for s, n in LENGTHS.items()}
    y[0][:, nk:2 * nk][40:45] = -60.0                     # gates of (with a lower bound of 0) next to nothing
    y[0][:, nk:2 * nk][60:90] = 25.0                      # and of 1: nothing is written, nothing lost
    fb = torch.randn(nk, generator=g) + 1.0
    low = 0.98 * torch.rand(nk, generator=g)
    low[::3] = 0.0
    w = 1 + 0.3 * torch.randn(nv, generator=g)
    want, last = {}, {}
    for s in LENGTHS:
        yy = y[s].double()
        want[s], last[s] = _plain_recurrence(yy[:, :nk], yy[:, nk:2 * nk] + fb.double(), yy[:, 2 * nk:], low.double(), H, D, Dv)
    for normed in (False, True):
        state = torch.full((4, nk * Dv + 4), float("nan"), device=DEV)
        for s in SLOT.values():
            state[s, :nk * Dv] = 0

        def call(rows, seq, portions, single):
            r = rows[0]
            chunks = None
            if chunk and not single:
                ch, po = o.recurrence_chunks(portions, chunk)
                chunks = (ch.to(DEV), po.to(DEV))
            kw = dict(norm_weight=w.to(DEV), norm_eps=1e-5, norm_dtype=torch.float32, single_rows=single) if normed else {}
            out = o.linear_recurrence(r[:, :nk], r[:, nk:2 * nk], r[:, 2 * nk:], state, seq, H, silu=True, forget_bias=fb.to(DEV),
                                      lower=low.to(DEV), chunks=chunks, **kw)
            return out.view(-1, H, Dv)

        got = _walk(call, [y])
        for s in LENGTHS:
            ref = want[s] if not normed else B.rms_norm(want[s], w.double().view(H, Dv), 1e-5)
            assert rel(got[s], ref) < 2e-5, (s, normed)
            assert rel(state[SLOT[s], :nk * Dv].view(H, D, Dv), last[s]) < 1e-5
        assert torch.isnan(state[1]).all() and torch.isnan(state[:, nk * Dv:]).all()


@pytest.mark.parametrize("chunk", [0, 16, 128])
def test_a_state_far_back_is_kept_or_forgotten(chunk):
    """One early token writes a large value while every later gate is 1 (or 0.99): hundreds of tokens on, a query along
    that channel reads it back; random inputs alone would bury a lost state under the recent tokens."""
    o = ops()
    H, D, Dv, n = 2, 16, 24, 400
    z = torch.full((n, H * D), 30.0)
    z[2, 5] = z[2, D + 5] = -30.0                         # the one token that writes
    z[3:, D + 5] = math.log(0.99 / 0.01)
    q = torch.zeros(n, H * D)
    q[n - 1, 5] = q[n - 1, D + 5] = 8.0
    v = torch.zeros(n, H * Dv)
    v[2] = torch.arange(H * Dv).float() + 1
    zero = torch.zeros(H * D)
    want, _ = _plain_recurrence(q.double(), z.double(), v.double(), zero.double(), H, D, Dv)
    assert float(want[-1, 0].abs().max()) > 100 and 0.1 < float(want[-1, 1].abs().max()) < 10
    y = torch.cat([q, z, v], dim=1)
    for cut in ((n,), (3, 200, 197), (1,) * 20 + (n - 20,), (2, 14, 16, 17, n - 49)):
        state = torch.zeros(1, H * D * Dv, device=DEV)
        outs, at = [], 0
        for m in cut:
            r = y[at:at + m].to(DEV)
            chunks = tuple(t.to(DEV) for t in o.recurrence_chunks([(0, m)], chunk)) if chunk else None
            outs.append(o.linear_recurrence(r[:, :H * D], r[:, H * D:2 * H * D], r[:, 2 * H * D:], state, i32([0] * m), H, silu=True,
                                            forget_bias=zero.to(DEV), lower=zero.to(DEV), chunks=chunks))
            at += m
        assert rel(torch.cat(outs), want) < 2e-5, cut


# ---- attention: window, soft cap, a 1 in the denominator ---------------------------------------------------------------
def _paged(k, v, P, g, dtype, Dc):
    """One request's keys and values in scattered pages (the value tiles transposed), zeros beyond a head's own numbers
    and behind the last key, NaN in every other page."""
    n, G = k.shape[0], k.shape[1]
    pages = (n + P - 1) // P + 3
    tab = torch.randperm(pages, generator=g)[:(n + P - 1) // P].tolist()
    cache = torch.full((pages, 2, G, P, Dc), float("nan"), dtype=dtype)
    for pg in tab:
        cache[pg] = 0
    for j in range(n):
        pg, off = tab[j // P], j % P
        cache[pg, 0, :, off, :k.shape[2]] = k[j].to(dtype)
        cache[pg, 1].view(G, Dc, P)[:, :v.shape[2], off] = v[j].to(dtype)
    return cache.to(DEV), torch.tensor([tab], dtype=torch.int32).to(DEV)


def _plain_attention(q, k, v, scale, cap, window):
    n, H, G = q.shape[0], q.shape[1], k.shape[1]
    i, j = torch.arange(n)[:, None], torch.arange(n)[None, :]
    seen = (j <= i) & (i - j < window)
    out = []
    for h in range(H):
        s = B.soft_cap(q[:, h].double() @ k[:, h // (H // G)].double().T * scale, cap)
        out.append(B.softmax_with_one(s.masked_fill(~seen, -math.inf)) @ v[:, h // (H // G)].double())
    return torch.stack(out, dim=1)


def _attend(q, cache, bt, scale, cap, window, rows, Dc, algo=0):
    """Rows of q [n, H, d] through ops.attention as the engine asks: a portion by tiles, a single row by the decode list."""
    o = ops()
    from qwen_engine_amd.parts.attention import prefill_tiles
    T, H = len(rows), q.shape[1]
    qp = torch.zeros(T, H, Dc, dtype=q.dtype)
    qp[:, :, :q.shape[2]] = q[rows]
    kw = {}
    if T == 1:
        kw = dict(dec_tokens=i32([0]), max_dec_position=rows[0], other_tokens=i32([]))
    else:
        tr = o.prefill_tile_rows(H, cache.shape[2])
        tiles = i32(prefill_tiles([(0, T)], tr)).view(-1, 2) if tr > 0 else None
        kw = dict(dec_tokens=i32([]), other_tokens=i32(list(range(T))), other_tiles=tiles, max_other_keys=rows[-1] + 1)
    return o.attention(qp.to(DEV), cache, i32(rows), i32([0] * T), bt, scale, window, sink=True, softcap=cap, algo=algo, **kw)


@pytest.mark.parametrize("dtype,tol", [(torch.float32, 1e-5), (torch.bfloat16, 1.5e-2)])
@pytest.mark.parametrize("hq,hkv,d,dv,window,P,n,cap", [
    (6, 2, 20, 12, 37, 8, 100, 4.0), (8, 2, 64, 64, 64, 16, 300, 8.0), (5, 5, 48, 64, 70, 16, 200, 40.0), (16, 4, 128, 128, 200, 16, 420, 2.0),
    (1, 1, 40, 80, 1, 4, 30, 3.0), (12, 1, 100, 128, 130, 32, 280, 30.0), (4, 4, 160, 16, 33, 16, 90, 5.0), (5, 5, 64, 64, 1000, 16, 333, 6.0)])
def test_attention_with_window_soft_cap_and_sink(dtype, tol, hq, hkv, d, dv, window, P, n, cap):
    from qwen_engine_amd.parts.attention import common_head_dim
    g = torch.Generator().manual_seed(hq * n)
    r = lambda *s: torch.randn(*s, generator=g)
    q, k, v = r(n, hq, d).to(dtype), r(n, hkv, d).to(dtype), r(n, hkv, dv).to(dtype)
    scale = 2.5 / math.sqrt(d)                             # (scores of several: a cap of 2 to 8 bends them)
    want = _plain_attention(q, k, v, scale, cap, window)
    Dc = common_head_dim(d, dv)
    cache, bt = _paged(k, v, P, g, dtype, Dc)
    got = _attend(q, cache, bt, scale, cap, window, list(range(n)), Dc)
    assert rel(got[:, :, :dv], want) < tol
    a, b = n // 3, n - 2
    assert rel(_attend(q, cache, bt, scale, cap, window, list(range(a, b)), Dc)[:, :, :dv], want[a:b]) < tol
    for p in sorted({0, min(window - 1, n - 1), min(window, n - 1), n // 2, n - 1}):
        assert rel(_attend(q, cache, bt, scale, cap, window, [p], Dc)[0, :, :dv], want[p]) < tol, p
        assert rel(_attend(q, cache, bt, scale, cap, window, [p], Dc, algo=1)[0, :, :dv], want[p]) < tol, p


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("d,window,n", [(64, 70, 200), (128, 144, 333), (16, 33, 90)])
def test_the_key_at_the_windows_edge_stands_out_and_the_one_behind_it_is_not_seen(dtype, d, window, n):
    """One key so large that its (capped) score carries the softmax: the output is its value while it is the window's
    last, and the rest's once the window has passed it; in a portion and alone."""
    g = torch.Generator().manual_seed(d)
    r = lambda *s: torch.randn(*s, generator=g) * 0.3
    hq, hkv, j = 4, 2, 40 if window < 100 else 100
    q, k, v = r(n, hq, d), r(n, hkv, d), r(n, hkv, d) * 3
    q[:, :, 3] = 8.0
    k[:, :, 3] = -8.0
    k[j, :, 3] = 8.0
    q, k, v = q.to(dtype), k.to(dtype), v.to(dtype)
    cache, bt = _paged(k, v, 16, g, dtype, max(d, 64))
    want = _plain_attention(q, k, v, 1.0, 30.0, window)
    last_in, first_out = j + window - 1, j + window
    near = lambda x, p: float((x[:, :d].double().cpu() - v[j].double().repeat_interleave(2, dim=0)).abs().max()) < 2e-2
    for rows in (list(range(n)), list(range(last_in - 1, first_out + 3))):
        got = _attend(q, cache, bt, 1.0, 30.0, window, rows, max(d, 64))
        assert near(got[rows.index(last_in)], j) and not near(got[rows.index(first_out)], j)
        assert float((got[rows.index(first_out)][:, :d].double().cpu() - want[first_out]).abs().max()) < 1e-3   # (all far below the added 1)
    assert near(_attend(q, cache, bt, 1.0, 30.0, window, [last_in], max(d, 64))[0], j)
    assert not near(_attend(q, cache, bt, 1.0, 30.0, window, [first_out], max(d, 64))[0], j)


def test_output_projection_partial_products_carry_the_bias_once():
    o = ops()
    g = torch.Generator().manual_seed(1)
    for M, N, K in ((1, 256, 512), (9, 200, 1024), (70, 512, 4096)):
        x, w, b = torch.randn(M, K, generator=g).bfloat16(), torch.randn(N, K, generator=g).bfloat16() * 0.05, torch.randn(N, generator=g) * 5
        want = x.double() @ w.double().T + b.double()
        splits = o.gemm_branch_splits(x.to(DEV), w.to(DEV)) or 2
        got = o.gemm(x.to(DEV), w.to(DEV), b.to(DEV), epilogue=o.EPI_PARTIAL, splits=splits)
        assert got.shape[0] == splits and rel(got.sum(0), want) < 1e-5, (M, N, K)


# ---- the mixture --------------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("T,E,top,transposed", [(9, 6, 2, False), (70, 16, 4, True), (5, 3, 3, False), (40, 4, 1, False), (3, 70, 5, False)])
def test_router_with_sigmoid_scores(T, E, top, transposed):
    g = torch.Generator().manual_seed(T + E)
    z = torch.randn(T, E, generator=g) * 2.0
    z[0] = -30.0 * torch.arange(E)                                 # sigmoids of 1/2, then of next to nothing: as they are
    z[1] = 40.0 + torch.arange(E)                                  # sigmoids that are all 1 in 32-bit
    dev = z.t().contiguous().to(DEV) if transposed else z.to(DEV)
    ids, w = ops().moe_route_biased(dev, None, top, 1.0, transposed=transposed, sigmoid=True)
    want_ids, want_w = B.route_sigmoid(z.double(), top)
    assert torch.equal(ids.cpu().long(), want_ids)
    assert rel(w, want_w) < 1e-6
    ids2, w2 = ops().moe_route_biased(dev, None, top, 2.5, transposed=transposed, sigmoid=True)
    assert torch.equal(ids2, ids) and rel(w2, 2.5 * want_w) < 1e-6


@pytest.mark.parametrize("dtype,tol", [(torch.float32, 3e-6), (torch.bfloat16, 1.5e-2)])
@pytest.mark.parametrize("T,E,top,Fd,W", [(5, 6, 2, 40, 128), (300, 8, 3, 160, 128), (600, 4, 2, 64, 128), (1, 3, 3, 32, 256), (2, 5, 1, 20, 70),
                                          (1500, 5, 1, 96, 64), (90, 16, 8, 96, 512), (33, 1, 1, 24, 96)])
def test_mixture_that_weighs_its_experts_inputs(dtype, tol, T, E, top, Fd, W):
    """The part itself on every path: the one-launch front, rows in place, the tiled grouped product, the vector units."""
    from qwen_engine_amd.config.spec import SigmoidMoESpec
    from qwen_engine_amd.parts import Runtime, build_part
    g = torch.Generator().manual_seed(T + E)
    r = lambda *s: torch.randn(*s, generator=g)
    w = {"router": (r(E, W) * 2.5 / math.sqrt(W)).bfloat16()}
    for e in range(E):
        w[f"e{e}.gate"], w[f"e{e}.up"], w[f"e{e}.down"] = [(m * 2.0 / math.sqrt(m.shape[-1])).bfloat16()
                                                          for m in (r(Fd, W), r(Fd, W), r(W, Fd))]
    rt = Runtime(torch.device(DEV), dtype)
    x = r(T, W).to(dtype)

    class Ctx:
        pass
    ctx = Ctx()
    ctx.rt = rt
    for weigh_input in (True, False):
        part = build_part(SigmoidMoESpec(num_experts=E, top=top, intermediate_size=Fd, weigh_input=weigh_input), W)
        part.load(w, rt)
        got = part.forward(x.to(DEV), ctx).sum(0)
        if weigh_input:
            want = B.mixture(x.double(), w, "", {"router": {"top": top}})
        else:
            ids, wts = B.route_sigmoid(x.double() @ w["router"].double().T, top)
            want = torch.stack([sum(wts[t, c] * B.expert(x[t:t + 1].double(), w, f"e{int(ids[t, c])}.")[0] for c in range(top))
                                for t in range(T)])
        if dtype == torch.float32:
            assert rel(got, want) < tol
        else:
            # (a router's close call may fall the other way in bfloat16: nearly every row agrees)
            err = (got.double().cpu() - want).abs().amax(dim=1) / float(want.abs().max())
            assert float((err > tol).float().mean()) <= 0.03, f"{int((err > tol).sum())} of {T} rows differ"
