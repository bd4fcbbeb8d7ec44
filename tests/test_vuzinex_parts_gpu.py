"""Each mechanism of the Vuzinex layers alone: the kernel against the plain implementation's function of the same
mechanism (or a few lines of 64-bit torch), in float32 and bfloat16."""
import math

import pytest
import torch
import torch.nn.functional as F

import qwen_engine_amd  # noqa: F401
from plain import vuzinex_plain as B

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
    """Feeds every request's rows through ``call(rows, table rows, portions, positions)`` in STEPS; each request's outputs in
    order.  A portion list is given to every call; single rows are recognised from it."""
    done = {s: 0 for s in LENGTHS}
    got = {s: [] for s in LENGTHS}
    for step in STEPS:
        rows, seq, pos, portions, at = [[] for _ in inputs], [], [], [], 0
        for s, n in step:
            for i, t in enumerate(inputs):
                rows[i].append(t[s][done[s]:done[s] + n])
            seq += [SLOT[s]] * n
            pos += range(done[s], done[s] + n)
            portions.append((at, n))
            at += n
        out = call([torch.cat(r).to(DEV) for r in rows], i32(seq), portions, i32(pos))
        at = 0
        for s, n in step:
            got[s].append(out[at:at + n].cpu())
            at += n
            done[s] += n
    assert done == LENGTHS
    return {s: torch.cat(v) for s, v in got.items()}


def _single(portions):
    return all(n == 1 for _, n in portions)


def _chunks(portions, length):
    """The chunk lists where some portion is long, as the engine asks; length 0: never."""
    if not length or max(n for _, n in portions) < 8:
        return None
    return tuple(t.to(DEV) for t in ops().recurrence_chunks(portions, length))


# ---- embedding of pairs ------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("H,V,buckets,a,b", [(96, 50, 17, 7, 13), (70, 31, 1, 3, 5), (1024, 200, 503, 1000003, 999983)])
def test_embedding_of_pairs(dtype, H, V, buckets, a, b):
    g = torch.Generator().manual_seed(H)
    table, pairs = torch.randn(V, H, generator=g).to(dtype), torch.randn(buckets + 1, H, generator=g).to(dtype)
    ids = {s: torch.randint(0, V, (n,), generator=g, dtype=torch.int32) for s, n in LENGTHS.items()}
    last = torch.full((5, 1), 12345, dtype=torch.int32, device=DEV)          # (what stands there before a request is not read)

    def call(rows, seq, portions, pos):
        return ops().embedding_pairs(rows[0], pos, seq, last, table.to(DEV), pairs.to(DEV), 1.7, a, b, single_rows=_single(portions))

    got = _walk(call, [ids])
    for s in LENGTHS:
        toks = ids[s].tolist()
        want = 1.7 * table[toks].double() + pairs[B.bigram_rows(toks, buckets, a, b)].double()
        assert rel(got[s], want) < 1e-6
        assert int(last[SLOT[s]]) == toks[-1]


# ---- the norms around a sublayer ---------------------------------------------------------------------------------------
@pytest.mark.parametrize("H", [64, 70, 96, 1024, 2052, 4096, 8192, 9000])
@pytest.mark.parametrize("kind", ["float32", "parts", "bfloat16", "bfloat16 parts"])
def test_branch_norm(H, kind):
    g = torch.Generator().manual_seed(H)
    T = 5
    dtype = torch.bfloat16 if kind.startswith("b") else torch.float32
    shape = (3, T, H) if "parts" in kind else (T, H)
    h, wb, w = torch.randn(T, H, generator=g) * 3, 1 + 0.3 * torch.randn(H, generator=g), 1 + 0.3 * torch.randn(H, generator=g)
    y = torch.randn(*shape, generator=g).to(torch.float32 if "parts" in kind else dtype)
    y[..., 2, :] = 0                                       # (a branch of zeros adds nothing: eps keeps it from the root of 0)
    total = y.double().sum(0) if "parts" in kind else y.double()
    want_h = h.double() + 0.7 * B.unit(1.9 * total, 1e-3) * wb.double()
    want = B.unit(want_h, 1e-5) * w.double()
    hd = h.to(DEV)
    rows = i32([4, 0, 2])
    got = ops().branch_norm(hd, y.to(DEV), wb.to(DEV), 1e-3, 0.7, w.to(DEV), 1e-5, dtype, scale=1.9, rows=rows)
    assert torch.equal(hd.cpu(), h) and rel(got, want[[4, 0, 2]]) < (1e-2 if dtype == torch.bfloat16 else 2e-6)
    got = ops().branch_norm(hd, y.to(DEV), wb.to(DEV), 1e-3, 0.7, w.to(DEV), 1e-5, dtype, scale=1.9)
    assert got.dtype == dtype and rel(got, want) < (1e-2 if dtype == torch.bfloat16 else 2e-6)
    assert rel(hd, want_h) < 2e-6
    hd = h.to(DEV)
    assert ops().branch_norm(hd, y.to(DEV), wb.to(DEV), 1e-3, 0.7, None, 0.0, dtype, scale=1.9) is None and rel(hd, want_h) < 2e-6


def test_branch_norm_of_many_rows():
    g = torch.Generator().manual_seed(1)
    h, y = torch.randn(700, 512, generator=g), torch.randn(700, 512, generator=g).bfloat16()
    w = torch.ones(512)
    want = h.double() + 0.5 * B.unit(y.double(), 1e-5)
    hd = h.to(DEV)
    got = ops().branch_norm(hd, y.to(DEV), w.to(DEV), 1e-5, 0.5, w.to(DEV), 1e-5, torch.bfloat16)
    assert rel(hd, want) < 2e-6 and rel(got, B.unit(want, 1e-5)) < 1e-2


# ---- attention: chunks, sinks, the gate, narrower values --------------------------------------------------------------
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


def _attend(q, cache, bt, scale, chunk, rows, Dc, dv, sink, gate, algo=0, out=None):
    """Rows of q [n, H, d] through ops.attention as the engine asks: a portion by tiles, a single row by the decode list."""
    o = ops()
    from qwen_engine_amd.parts.attention import prefill_tiles
    T, H = len(rows), q.shape[1]
    qp = torch.zeros(T, H, Dc, dtype=q.dtype)
    qp[:, :, :q.shape[2]] = q[rows]
    if T == 1:
        kw = dict(dec_tokens=i32([0]), max_dec_position=rows[0], other_tokens=i32([]))
    else:
        tr = o.prefill_tile_rows(H, cache.shape[2])
        tiles = i32(prefill_tiles([(0, T)], tr)).view(-1, 2) if tr > 0 else None
        kw = dict(dec_tokens=i32([]), other_tokens=i32(list(range(T))), other_tiles=tiles, max_other_keys=rows[-1] + 1)
    gd = None
    if gate is not None:                                   # (columns of wider rows)
        wide = torch.full((T, gate.shape[1] + 8), float("nan"), dtype=gate.dtype)
        wide[:, 4:4 + gate.shape[1]] = gate[rows]
        gd = wide.to(DEV)[:, 4:4 + gate.shape[1]]
    return o.attention(qp.to(DEV), cache, i32(rows), i32([0] * T), bt, scale, 0, chunk=chunk or 0, v_dim=dv, gate=gd,
                       sink=False if sink is None else sink.to(DEV), algo=algo, out=out, **kw)


CASES = [(6, 2, 20, 12, 37, 8, 100), (8, 2, 64, 64, 64, 16, 300), (5, 5, 48, 64, None, 16, 200), (16, 4, 128, 128, 200, 16, 420),
         (1, 1, 40, 80, 1, 4, 30), (12, 1, 96, 96, 96, 32, 280), (4, 4, 160, 16, 33, 16, 90), (3, 3, 10, 6, 21, 2, 70), (6, 2, 64, 50, None, 16, 1300)]


@pytest.mark.parametrize("dtype,tol", [(torch.float32, 1e-5), (torch.bfloat16, 1.5e-2)])
@pytest.mark.parametrize("with_sink,gate_type", [(True, None), (False, "own"), (True, torch.float32), (False, None)])
@pytest.mark.parametrize("hq,hkv,d,dv,chunk,P,n", CASES)
def test_attention_in_chunks_with_sinks_and_a_gate(dtype, tol, with_sink, gate_type, hq, hkv, d, dv, chunk, P, n):
    from qwen_engine_amd.parts.attention import common_head_dim
    g = torch.Generator().manual_seed(hq * n)
    r = lambda *s: torch.randn(*s, generator=g)
    q, k, v = r(n, hq, d).to(dtype), r(n, hkv, d).to(dtype), r(n, hkv, dv).to(dtype)
    sink = 3 * r(hq) if with_sink else None
    gate = (2 * r(n, hq * dv)).to(dtype if gate_type == "own" else gate_type) if gate_type is not None else None
    scale = 1.5 / math.sqrt(d)
    want = B.attend(q.double(), k.double(), v.double(), scale, B.chunk_mask(n, chunk), None if sink is None else sink.double())
    if gate is not None:
        want = want * torch.sigmoid(gate.double())
    Dc = common_head_dim(d, dv)
    cache, bt = _paged(k, v, P, g, dtype, Dc)
    assert rel(_attend(q, cache, bt, scale, chunk, list(range(n)), Dc, dv, sink, gate), want) < tol
    a, b = n // 3, n - 2
    # into columns of wider rows, the others untouched
    wide = torch.full((b - a, hq * dv + 12), 7.0, dtype=dtype, device=DEV)
    _attend(q, cache, bt, scale, chunk, list(range(a, b)), Dc, dv, sink, gate, out=wide[:, 8:8 + hq * dv])
    assert rel(wide[:, 8:8 + hq * dv], want[a:b]) < tol and bool((wide[:, :8] == 7).all()) and bool((wide[:, 8 + hq * dv:] == 7).all())
    c = chunk or n
    for p in sorted({0, min(c - 1, n - 1), min(c, n - 1), n // 2, n - 1}):
        for algo in (0, 1):
            assert rel(_attend(q, cache, bt, scale, chunk, [p], Dc, dv, sink, gate, algo=algo)[0], want[p]) < tol, (p, algo)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("d,chunk,n", [(64, 70, 200), (128, 144, 333), (16, 33, 90)])
def test_the_first_key_of_a_chunk_stands_out_and_the_last_of_the_one_before_is_not_seen(dtype, d, chunk, n):
    """Two keys so large that their scores carry the softmax: the last of a chunk and the first of the next.  Every row of
    a chunk gives the value of the large key it sees; with a sink far above every score nothing is left of it."""
    g = torch.Generator().manual_seed(d)
    r = lambda *s: torch.randn(*s, generator=g) * 0.3
    hq, hkv = 4, 2
    q, k, v = r(n, hq, d), r(n, hkv, d), r(n, hkv, d) * 3
    q[:, :, 3] = 8.0
    k[:, :, 3] = -8.0
    k[chunk - 1, :, 3] = k[chunk, :, 3] = 8.0
    q, k, v = q.to(dtype), k.to(dtype), v.to(dtype)
    cache, bt = _paged(k, v, 16, g, dtype, max(d, 64))
    near = lambda x, p: float((x.view(hq, d).double().cpu() - v[p].double().repeat_interleave(2, dim=0)).abs().max()) < 2e-2
    none = torch.zeros(hq)
    for rows in (list(range(n)), list(range(chunk - 2, chunk + 3))):
        got = _attend(q, cache, bt, 1.0, chunk, rows, max(d, 64), d, none, None)
        assert near(got[rows.index(chunk - 1)], chunk - 1) and near(got[rows.index(chunk)], chunk) and near(got[rows.index(chunk + 2)], chunk)
        assert float(_attend(q, cache, bt, 1.0, chunk, rows, max(d, 64), d, none + 200.0, None).abs().max()) < 1e-6
    for p, sees in ((chunk - 1, chunk - 1), (chunk, chunk), (chunk + 1, chunk), (2 * chunk - 1, chunk)):
        assert near(_attend(q, cache, bt, 1.0, chunk, [p], max(d, 64), d, none, None)[0], sees)
    alone = _attend(q, cache, bt, 1.0, chunk, [2 * chunk], max(d, 64), d, none, None)[0]
    assert not near(alone, chunk) and float(alone.abs().max()) < 1e-3          # (the third chunk: only its own, far below the sink)


# ---- between the projection and attention ----------------------------------------------------------------------------
@pytest.mark.parametrize("src,dst", [(torch.float32, torch.float32), (torch.bfloat16, torch.bfloat16), (torch.float32, torch.bfloat16)])
@pytest.mark.parametrize("hq,hkv,d,dv,rot,T,norm", [(6, 2, 20, 12, 12, 9, True), (4, 4, 64, 64, 64, 600, True), (1, 1, 32, 48, 0, 3, False),
                                                    (8, 2, 96, 96, 96, 33, True), (5, 5, 6, 10, 2, 7, False)])
def test_norm_rotation_of_neighbouring_pairs_and_cache_write(src, dst, hq, hkv, d, dv, rot, T, norm):
    from qwen_engine_amd.parts.attention import common_head_dim
    o = ops()
    g = torch.Generator().manual_seed(hq * T)
    r = lambda *s: torch.randn(*s, generator=g)
    n = hq * d + hkv * (d + dv)
    y = r(T, n + 5).to(src)
    qw, kw = 1 + 0.3 * r(d), 1 + 0.3 * r(d)
    pos = torch.randint(0, 3000, (T,), generator=g)
    freq, gain = B.yarn(300.0, rot, dict(factor=3.0, original=200, fast=8.0, slow=1.0)) if rot else ([], 1.0)
    f32 = torch.tensor(freq, dtype=torch.float32)
    P, Dc = 8, common_head_dim(d, dv)
    pages = (T + P - 1) // P + 1
    slots = torch.randperm(pages * P, generator=g)[:T].to(torch.int32)
    slots[T // 2] = -1                                     # (a row that writes nowhere)
    cache = torch.full((pages, 2, hkv, P, Dc), 9.0, dtype=dst, device=DEV)
    q = o.qkv_norm_store(y.to(DEV)[:, :n], hq, hkv, d, dv, cache, slots.to(DEV), qk_norm=o.QK_NORM_HEAD if norm else o.QK_NORM_NONE,
                         q_weight=qw.to(DEV) if norm else None, k_weight=kw.to(DEV) if norm else None, qk_eps=1e-5, positions=i32(pos.tolist()),
                         inv_freq=f32.to(DEV) if rot else None, rot_pairs=True, rot_gain=gain)
    yd = y.double()
    qs, ks, vs = yd[:, :hq * d].view(T, hq, d), yd[:, hq * d:(hq + hkv) * d].view(T, hkv, d), yd[:, (hq + hkv) * d:n].view(T, hkv, dv)
    if norm:
        qs, ks = B.unit(qs, 1e-5) * qw.double(), B.unit(ks, 1e-5) * kw.double()
    qs, ks = (B.rotate_neighbours(t, pos, f32.double().tolist(), gain) for t in (qs, ks))
    tol = 1e-2 if dst == torch.bfloat16 else 5e-4          # (angles of some thousands in 32-bit)
    assert rel(q[:, :, :d], qs) < tol and float(q[:, :, d:].abs().float().sum()) == 0 and q.dtype == dst
    for t in range(T):
        if slots[t] < 0:
            continue
        pg, off = int(slots[t]) // P, int(slots[t]) % P
        assert rel(cache[pg, 0, :, off, :d], ks[t]) < tol and rel(cache[pg, 1].view(hkv, Dc, P)[:, :dv, off], vs[t]) < tol
    assert int((cache == 9.0).all(dim=-1)[:, 0, 0].sum()) == pages * P - (T - 1)


# ---- the recurrences -------------------------------------------------------------------------------------------------
SIZES = [(3, 12, 20), (2, 28, 16), (2, 64, 64), (3, 32, 128), (1, 3, 7), (2, 22, 5), (2, 160, 40), (1, 16, 144), (4, 48, 48), (2, 128, 96), (1, 256, 33), (2, 128, 64), (3, 100, 33)]


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("length", [0, 16, 64])
@pytest.mark.parametrize("H,D,Dv", SIZES)
def test_gated_linear_recurrence(dtype, length, H, D, Dv):
    """Decays per channel from a low rank, the norm per head, the silu gate and the scale behind them."""
    o = ops()
    g = torch.Generator().manual_seed(H * D + Dv)
    r = lambda *s: torch.randn(*s, generator=g)
    R, tau = 5, 3.0
    nk, nv = H * D, H * Dv
    y = {s: r(n, 2 * nk + 2 * nv + R).to(dtype) for s, n in LENGTHS.items()}
    w2, b2, nw = r(nk, R), 2 + 2 * r(nk), (1 + 0.3 * r(Dv)).repeat(H)
    w2t = w2.t().contiguous()
    state = torch.zeros(5, H * D * Dv + 8, device=DEV)
    st = state[:, 4:]

    def call(rows, seq, portions, pos):
        x = rows[0]
        out = torch.full((x.shape[0], nv + 6), 5.0, device=DEV, dtype=dtype)
        o.linear_recurrence(x[:, :nk], x[:, nk:2 * nk], x[:, 2 * nk:2 * nk + nv], st, seq, H, q_scale=D ** -0.5,
                            low_rank=(x[:, 2 * nk + 2 * nv:], w2t.to(DEV), b2.to(DEV), tau), chunks=_chunks(portions, length), norm_weight=nw.to(DEV),
                            norm_eps=1e-5, norm_dtype=dtype, single_rows=_single(portions), gate=x[:, 2 * nk + nv:2 * nk + 2 * nv],
                            gate_act=o.GATE_SILU, y_scale=0.6, out=out[:, 2:2 + nv])
        assert bool((out[:, :2] == 5).all()) and bool((out[:, 2 + nv:] == 5).all())
        return out[:, 2:2 + nv]

    got = _walk(call, [y])
    for s in LENGTHS:
        x = y[s].double()
        T = x.shape[0]
        alpha = torch.exp(B.log_sigmoid(x[:, 2 * nk + 2 * nv:] @ w2.double().T + b2.double()) / tau).view(T, H, D)
        want, S = B.decayed_outer(x[:, :nk].view(T, H, D) * D ** -0.5, x[:, nk:2 * nk].view(T, H, D), x[:, 2 * nk:2 * nk + nv].view(T, H, Dv), alpha)
        want = 0.6 * B.unit(want, 1e-5).reshape(T, nv) * nw.double() * B.silu(x[:, 2 * nk + nv:2 * nk + 2 * nv])
        assert rel(got[s], want) < (1.5e-2 if dtype == torch.bfloat16 else 2e-5), s
        assert rel(st[SLOT[s], :H * D * Dv], S.reshape(-1)) < 2e-5
    assert float(state[:, :4].abs().max()) == 0 and float(state[:, 4 + H * D * Dv:].abs().max()) == 0 and float(state[4].abs().max()) == 0


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("length", [0, 16, 64])
@pytest.mark.parametrize("H,D,Dv", SIZES)
def test_matrix_memory(dtype, length, H, D, Dv):
    """Gates, running maximum, state, normaliser, the norm per head and the sigmoid gate behind them."""
    o = ops()
    g = torch.Generator().manual_seed(H * D + Dv + 1)
    r = lambda *s: torch.randn(*s, generator=g)
    nk, nv, cap = H * D, H * Dv, 7.0
    y = {s: r(n, 2 * nk + 2 * nv).to(dtype) for s, n in LENGTHS.items()}
    z = {s: 4 * r(n, 2 * H + 3) for s, n in LENGTHS.items()}
    ib, fb, nw = 2 * r(H), 2 + 2 * r(H), 1 + 0.3 * r(nv)
    at = o.recurrence_state_numbers(H, D, Dv, normaliser=True)
    state = torch.zeros(5, (at + H + 3) // 4 * 4, device=DEV)

    def call(rows, seq, portions, pos):
        x, gates = rows
        return o.linear_recurrence(x[:, :nk], x[:, nk:2 * nk], x[:, 2 * nk:2 * nk + nv], state, seq, H, q_scale=D ** -0.5,
                                   gates=(gates[:, 1:1 + 2 * H], ib.to(DEV), fb.to(DEV), cap, at), chunks=_chunks(portions, length),
                                   norm_weight=nw.to(DEV), norm_eps=1e-5, norm_dtype=dtype, single_rows=_single(portions),
                                   gate=x[:, 2 * nk + nv:], gate_act=o.GATE_SIGMOID)

    got = _walk(call, [y, z])
    for s in LENGTHS:
        x, zz = y[s].double(), z[s].double()[:, 1:1 + 2 * H]
        T = x.shape[0]
        i = cap * torch.tanh((zz[:, :H] + ib.double()) / cap)
        f = B.log_sigmoid(cap * torch.tanh((zz[:, H:] + fb.double()) / cap))
        raw, (S, n, m) = B.matrix_memory(x[:, :nk].view(T, H, D) * D ** -0.5, x[:, nk:2 * nk].view(T, H, D), x[:, 2 * nk:2 * nk + nv].view(T, H, Dv), i, f)
        want = B.unit(raw, 1e-5).reshape(T, nv) * nw.double() * B.sigmoid(x[:, 2 * nk + nv:])
        assert rel(got[s], want) < (1.5e-2 if dtype == torch.bfloat16 else 1e-4), s
        row = state[SLOT[s]]
        assert rel(row[:nk * Dv], S.reshape(-1)) < 3e-5 and rel(row[at:at + H], m) < 1e-5
        for z_ in range((Dv + 63) // 64):                  # (every copy of the normaliser)
            assert rel(row[nk * Dv + z_ * nk:nk * Dv + (z_ + 1) * nk], n.reshape(-1)) < 3e-5


@pytest.mark.parametrize("parts", [1, 3])
@pytest.mark.parametrize("T", [1, 5, 600, 2500, 4700])
def test_memory_gates_over_portions(T, parts):
    """The running maximum over many rows (a scan), against the token-by-token recursion, also from partial products, and
    from a maximum that an earlier step left; gates near -cap keep the start of 0 in play."""
    o = ops()
    g = torch.Generator().manual_seed(T)
    H, cap = 5, 12.0
    z = 8 * torch.randn(parts, T, 2 * H, generator=g)
    ib, fb = torch.tensor([0.0, -30.0, 30.0, 5.0, -5.0]), torch.tensor([0.0, 8.0, 5.0, -9.0, 20.0])
    m0 = torch.tensor([0.0, 0.0, 3.0, -1.0, 11.0])
    rm = torch.zeros(3, 8, device=DEV)
    rm[1, 2:2 + H] = m0.to(DEV)
    chunks = tuple(t.to(DEV) for t in o.recurrence_chunks([(0, T)], 64)) if T >= 8 else None
    zz = z.to(DEV) if parts > 1 else z[0].to(DEV)
    got = o.memory_gates(zz, ib.to(DEV), fb.to(DEV), cap, rm[:, 2:2 + H], i32([1] * T), chunks=chunks)
    zs = z.double().sum(0)
    i = cap * torch.tanh((zs[:, :H] + ib.double()) / cap)
    f = B.log_sigmoid(cap * torch.tanh((zs[:, H:] + fb.double()) / cap))
    m, rows = m0.double(), []
    for t in range(T):
        n = torch.maximum(f[t] + m, i[t])
        rows.append(torch.cat([torch.exp(f[t] + m - n), torch.exp(i[t] - n), torch.exp(-n)]))
        m = n
    want = torch.stack(rows)
    for c in range(3):
        a, b = got[:, c].double().cpu(), want[:, c * H:(c + 1) * H]
        assert float(((a - b).abs() / (b.abs() + 1e-3)).max()) < 5e-5, c
    assert rel(rm[1, 2:2 + H], m) < 1e-5 and float(rm[0].abs().max()) == 0


@pytest.mark.parametrize("low_type", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("T,N,R,tau", [(1, 96, 16, 16.0), (20, 300, 7, 1.0), (130, 512, 40, 5.0)])
def test_decays_through_a_low_rank(low_type, T, N, R, tau):
    g = torch.Generator().manual_seed(T)
    y = (2 * torch.randn(T, R + 9, generator=g)).to(low_type)
    w, b = torch.randn(N, R, generator=g), torch.cat([torch.tensor([-60.0, 60.0, 0.0]), torch.randn(N - 3, generator=g)])
    got = ops().low_rank_decay(y.to(DEV)[:, 4:4 + R], w.t().contiguous().to(DEV), b.to(DEV), tau)
    want = torch.sigmoid(y[:, 4:4 + R].double() @ w.double().T + b.double()) ** (1 / tau)
    assert float(((got.double().cpu() - want).abs() / (want + 1e-12)).max()) < 2e-5


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("length", [0, 16, 64])
@pytest.mark.parametrize("H,Dv,N,G,taps,parts", [(6, 10, 14, 2, 3, 3), (4, 16, 20, 1, 4, 1), (4, 64, 32, 1, 4, 1), (3, 8, 8, 3, 1, 1), (5, 6, 7, 1, 6, 2),
                                                 (2, 15, 9, 2, 2, 5), (8, 64, 128, 2, 4, 2), (2, 144, 144, 1, 5, 1), (2, 96, 3, 1, 4, 1)])
def test_state_space(dtype, length, H, Dv, N, G, taps, parts):
    """Convolution, step sizes, recurrence, skip, gate and norm, as the mixer strings them together."""
    o = ops()
    g = torch.Generator().manual_seed(H * Dv + N)
    r = lambda *s: torch.randn(*s, generator=g)
    inner, gn = H * Dv, G * N
    C = inner + 2 * gn
    y = {s: r(n, inner + C).to(dtype) for s, n in LENGTHS.items()}
    z = {s: r(n, H + 2) for s, n in LENGTHS.items()}
    cw, cb, db, A, D, nw = 0.5 * r(C, taps), 0.4 * r(C), r(H) - 1.5, 0.4 * r(H), r(H), 1 + 0.3 * r(inner)
    off = (H * N * Dv + 3) // 4 * 4
    state = torch.zeros(5, (off + (taps - 1) * C + 3) // 4 * 4, device=DEV)

    def call(rows, seq, portions, pos):
        x, dt = rows
        chunks = _chunks(portions, length)
        xbc, steps = o.conv_steps(x[:, inner:], cw.t().contiguous().to(DEV), cb.to(DEV), state[:, off:], seq, dt=dt[:, 1:1 + H], dt_bias=db.to(DEV),
                                  a_log=A.to(DEV), single_rows=_single(portions), chunks=chunks)
        out = o.linear_recurrence(xbc[:, inner + gn:], xbc[:, inner:inner + gn], xbc[:, :inner], state, seq, H, steps=steps, k_heads=G,
                                  chunks=chunks, single_rows=_single(portions))
        return o.skip_gate_norm(out, xbc[:, :inner], D.to(DEV), x[:, :inner], nw.to(DEV), 1e-5, parts, dtype)

    got = _walk(call, [y, z])
    for s in LENGTHS:
        x = y[s].double()
        T = x.shape[0]
        xbc = B.silu(B.causal_convolution(x[:, inner:], cw.double(), cb.double()))
        if dtype == torch.bfloat16:
            xbc = xbc.to(dtype).double()                   # (the convolved rows are activations)
        xs, Bm, Cm = xbc[:, :inner].view(T, H, Dv), xbc[:, inner:inner + gn].view(T, G, N), xbc[:, inner + gn:].view(T, G, N)
        want, S = B.state_space(xs, Bm, Cm, B.softplus(z[s].double()[:, 1:1 + H] + db.double()), A.double(), D.double())
        want = want.reshape(T, inner) * B.silu(x[:, :inner])
        want = B.unit(want.view(T, parts, inner // parts), 1e-5).reshape(T, inner) * nw.double()
        assert rel(got[s], want) < (2.5e-2 if dtype == torch.bfloat16 else 3e-5), s
        assert rel(state[SLOT[s], :H * N * Dv], S.reshape(-1)) < (1e-2 if dtype == torch.bfloat16 else 3e-5)
        if taps > 1:
            tail = torch.cat([torch.zeros(taps - 1, C, dtype=torch.float64), x[:, inner:]])[-(taps - 1):]
            assert torch.equal(state[SLOT[s], off:off + (taps - 1) * C].view(taps - 1, C).double().cpu(), tail)


def test_step_sizes_from_partial_products():
    o = ops()
    g = torch.Generator().manual_seed(3)
    dt = torch.randn(4, 11, 6, generator=g)
    db, A = torch.randn(6, generator=g), torch.randn(6, generator=g)
    x = torch.randn(11, 8, generator=g)
    _, steps = o.conv_steps(x.to(DEV), torch.ones(1, 8, device=DEV), torch.zeros(8, device=DEV), None, i32([0] * 11), dt=dt.to(DEV),
                            dt_bias=db.to(DEV), a_log=A.to(DEV))
    want = B.softplus(dt.double().sum(0) + db.double())
    assert rel(steps[:, 1], want) < 1e-6 and rel(steps[:, 0], torch.exp(-torch.exp(A.double()) * want)) < 1e-6


@pytest.mark.parametrize("mode", ["gated", "memory", "steps"])
def test_chunks_of_every_length_and_strong_decays_agree_with_row_by_row(mode):
    """Portions cut at odd places into chunks of 16 and 64, decays down to exp(-40) in a row: the chunked kernels against
    the plain recurrence."""
    o = ops()
    H, D, Dv, T = 2, 40, 72, 210
    g = torch.Generator().manual_seed(5)
    r = lambda *s: torch.randn(*s, generator=g)
    q, k, v = r(T, H * D), r(T, H * D), r(T, H * Dv)
    lf = -torch.rand(T, H * D if mode == "gated" else H, generator=g) * 0.2
    lf[torch.rand(T, generator=g) < 0.1] = -40.0           # (all is forgotten at once)
    write, floor = torch.rand(T, H, generator=g), torch.rand(T, H, generator=g)
    qd, kd, vd = q.double().view(T, H, D), k.double().view(T, H, D), v.double().view(T, H, Dv)
    keep = torch.exp(lf.double())
    S, n = torch.zeros(H, D, Dv, dtype=torch.float64), torch.zeros(H, D, dtype=torch.float64)
    want = torch.zeros(T, H, Dv, dtype=torch.float64)
    for t in range(T):
        a = keep[t].view(H, D, 1) if mode == "gated" else keep[t].view(H, 1, 1)
        kk = kd[t] if mode == "gated" else kd[t] * write[t].double()[:, None]
        S = a * S + kk[:, :, None] * vd[t][:, None, :]
        n = a[:, :, 0] * n + kk
        want[t] = (S * qd[t][:, :, None]).sum(1)
        if mode == "memory":
            want[t] /= (torch.maximum((n * qd[t]).sum(-1).abs(), floor[t].double()) + 1e-6)[:, None]
    kw = {"gated": dict(decays=keep.float().to(DEV)), "steps": dict(steps=torch.stack([keep[:, :H].float(), write], 1).to(DEV)),
          "memory": dict(steps=torch.stack([keep[:, :H].float(), write, floor], 1).to(DEV), normaliser=True)}[mode]
    for cuts in ([T], [64, 1, 145], [17, 16, 15, 2, 160], [100, 110]):
        for length in (16, 64):
            state = torch.zeros(1, o.recurrence_state_numbers(H, D, Dv, normaliser=mode == "memory"), device=DEV)
            outs, at = [], 0
            for m in cuts:
                part = {key: (val[at:at + m].contiguous() if torch.is_tensor(val) else val) for key, val in kw.items()}
                chunks = tuple(t.to(DEV) for t in o.recurrence_chunks([(0, m)], length))
                x = torch.cat([q, k, v], dim=1)[at:at + m].to(DEV)
                outs.append(o.linear_recurrence(x[:, :H * D], x[:, H * D:2 * H * D], x[:, 2 * H * D:], state, i32([0] * m), H, chunks=chunks, **part))
                at += m
            err = (torch.cat(outs).double().cpu() - want).abs().amax(dim=2) / want.abs().amax(dim=2).clamp(min=1e-3)
            assert float(err.quantile(0.99)) < 1e-4 and rel(torch.cat(outs), want) < 5e-5, (cuts, length)


# ---- the feed-forward's products with biases -----------------------------------------------------------------------
@pytest.mark.parametrize("dtype,tol", [(torch.float32, 1e-5), (torch.bfloat16, 2e-2)])
@pytest.mark.parametrize("inter", [96, 40])
@pytest.mark.parametrize("T", [1, 7, 40, 300])
def test_gated_feed_forward_with_biases(dtype, tol, inter, T):
    from qwen_engine_amd.config.spec import SwiGLUSpec
    from qwen_engine_amd.parts import Runtime, build_part
    g = torch.Generator().manual_seed(T + inter)
    W = 128
    w = {n: (torch.randn(*s, generator=g) * 1.3 / math.sqrt(s[-1])).to(dtype) for n, s in (("gate", (inter, W)), ("up", (inter, W)), ("down", (W, inter)))}
    w.update({n + ".b": torch.randn(m, generator=g).to(dtype) for n, m in (("gate", inter), ("up", inter), ("down", W))})
    spec = SwiGLUSpec(intermediate_size=inter, names=("gate", "up", "down"), bias=True)
    part = build_part(spec, W)
    part.load(w, Runtime(torch.device(DEV), dtype))
    x = torch.randn(T, W, generator=g).to(dtype)
    y = part.forward(x.to(DEV), None)
    y = y.float().sum(0) if y.dim() == 3 else y
    d = {n: t.double() for n, t in w.items()}
    want = F.linear(F.silu(F.linear(x.double(), d["gate"], d["gate.b"])) * F.linear(x.double(), d["up"], d["up.b"]), d["down"], d["down.b"])
    assert rel(y, want) < tol


@pytest.mark.parametrize("tile", [64, 65, 128, 256, 512])
@pytest.mark.parametrize("M,inter", [(300, 96), (70, 288)])
def test_biases_in_the_silu_epilogue_of_every_tile(tile, M, inter):
    o = ops()
    g = torch.Generator().manual_seed(tile)
    r = lambda *s: torch.randn(*s, generator=g)
    x, gate, up = r(M, 128).bfloat16(), (r(inter, 128) / 11).bfloat16(), (r(inter, 128) / 11).bfloat16()
    bg, bu = r(inter), r(inter)
    bias = o.interleave_gate_up(bg.view(-1, 1), bu.view(-1, 1)).view(-1)
    y = o.gemm(x.to(DEV), o.interleave_gate_up(gate, up).to(DEV), bias.to(DEV), epilogue=o.EPI_SILU_MUL_IL, algo=o.ALGO_TILE + tile)
    want = F.silu(x.double() @ gate.double().T + bg.double()) * (x.double() @ up.double().T + bu.double())
    assert rel(y, want) < 1e-2


@pytest.mark.parametrize("T", [1, 40, 65, 200])
@pytest.mark.parametrize("dtype,tol", [(torch.float32, 1e-5), (torch.bfloat16, 1e-2)])
def test_two_mixers_read_one_product_and_leave_one_row(T, dtype, tol):
    """The joint products of mixers side by side: columns, biases and the 32-bit columns where they belong, a row filled up to
    a multiple of 32 with zeros."""
    from qwen_engine_amd.parts import Runtime
    from qwen_engine_amd.parts.projected import InputProducts, OutputProduct
    g = torch.Generator().manual_seed(T)
    r = lambda *s: torch.randn(*s, generator=g)
    rt = Runtime(torch.device(DEV), dtype)
    K = 512
    a, b, c = (r(n, K).to(dtype) / 20 for n in (50, 70, 30))
    bias, g1, g2 = r(70).to(dtype), r(6, K).to(dtype) / 20, r(4, K).to(dtype) / 20
    ins = InputProducts([([(a, None), (b, bias)], []), ([(c, None)], [g1, g2])], rt)
    x = r(T, K).to(dtype)
    (y1, n1), (y2, n2) = ins.run(x.to(DEV), rt)
    xd = x.double()
    assert n1 is None and rel(y1, torch.cat([xd @ a.double().T, xd @ b.double().T + bias.double()], 1)) < tol and rel(y2, xd @ c.double().T) < tol
    n2 = n2.float().sum(0) if n2.dim() == 3 else n2
    assert n2.dtype == torch.float32 and rel(n2, xd @ torch.cat([g1, g2]).double().T) < 1e-5
    out = OutputProduct([a.t().contiguous()[:64], b.t().contiguous()[:64]], rt)
    o = out.rows(T, rt, torch.device(DEV))
    assert o.shape == (T, 128) and out.cols == [(0, 50), (50, 120)] and float(o[:, 120:].float().abs().max()) == 0
    o[:, :120] = r(T, 120).to(dtype).to(DEV)
    y = out.run(o)
    y = y.float().sum(0) if y.dim() == 3 else y
    od = o.double().cpu()
    assert rel(y, od[:, :50] @ a.double()[:, :64] + od[:, 50:120] @ b.double()[:, :64]) < tol
