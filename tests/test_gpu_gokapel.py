"""The Gokapel family on the gfx950 kernels: each op against its plain fp32
form, whole models against the oracle, in bf16 and in 32-bit."""
import io
import json

import numpy as np
import pytest
import torch

import gokapel_oracle as oracle
from gokapel_helpers import (MODELS, close, load, make, make_engine, portions,
                             rel_err, run_cut, tokens_of, write_checkpoint)
from runbooks_amd import ops
from runbooks_amd.models.ragged import StepPlan
from runbooks_amd.ops import delta as DR
from runbooks_amd.ops import min_gru as MG
from runbooks_amd.ops import moe as ME
from runbooks_amd.ops import qkv as QK
from runbooks_amd.ops import shared_kv as SK
from runbooks_amd.ops import streams as ST

pytestmark = pytest.mark.gpu

DEV = "cuda:0"
BF, F32 = torch.bfloat16, torch.float32
BATCHES = {"short": [(1, 0, 0), (1, 100, 0), (1, 15, 0), (2, 300, 16),
                     (1, 1500, 0), (7, 33, 0)],
           "mixed": [(1, 640, 0), (100, 0, 0), (3, 70, 0), (33, 90, 16),
                     (200, 500, 0), (700, 0, 0)]}


def operand_rows(swz, T):
    """Rows of a decode-GEMM operand."""
    return swz.view(-1, 2, 32, 8).permute(2, 0, 1, 3).reshape(32, -1)[:T]


def relative(a, ref):
    a, ref = a.float().cpu(), ref.float()
    return float((a - ref).abs().max() / ref.abs().max().clamp(min=1e-20))


@pytest.mark.parametrize("T,s,D", [(1, 1, 64), (7, 3, 200), (32, 4, 256),
                                   (33, 2, 90), (300, 4, 1024), (5, 7, 2560),
                                   (2, 16, 40), (3, 5, 33)])
@pytest.mark.parametrize("dtype", [BF, F32])
def test_streams_take_a_result_and_give_the_next_input(T, s, D, dtype):
    g = torch.Generator().manual_seed(0)
    r = lambda *n: torch.randn(*n, generator=g)  # noqa: E731
    x, inp, norm = r(T, s, D), r(s), r(2 * D + 1)
    y = r(T, D + 24).to(dtype)
    join = ST.pack_join(r(D), r(D), r(s), r(s, s) / s ** 0.5, 0.7)
    operand = dtype == BF and T <= 32
    tol = 2e-2 if dtype == BF else 2e-5
    for delta, extra in ((None, None), (r(T, D), None), (r(3, T, D), r(T, D)),
                         (r(T, D), r(2, T, D))):
        res = {}
        for dev in ("cpu", DEV):
            to = lambda t: None if t is None else t.to(dev)  # noqa: E731
            xx = x.to(dev).clone()
            p = None if delta is None else ops.Pending(
                to(delta), to(extra), to(y), 16, to(join))
            h = ops.streams_norm(xx, p, to(inp), to(norm), dtype,
                                 operand=operand and dev == DEV)
            assert h.dtype == dtype and h.shape == (T, -(-D // 32) * 32)
            res[dev] = (xx, h)
        assert relative(res[DEV][0], res["cpu"][0]) < 2e-5
        assert relative(res[DEV][1], res["cpu"][1]) < tol
        if operand:
            assert torch.equal(operand_rows(res[DEV][1]._rb_swz, T),
                               res[DEV][1])


@pytest.mark.parametrize("T,ff", [(1, 32), (32, 416), (33, 416), (300, 1024)])
@pytest.mark.parametrize("dtype", [BF, F32])
def test_squared_relu(T, ff, dtype):
    y = torch.randn(T, ff + 40, generator=torch.Generator().manual_seed(0)
                    ).to(dtype)
    operand = dtype == BF and T <= 32
    out = ops.squared_relu(y.to(DEV), ff, operand)
    ref = torch.relu(y[:, :ff].float()) ** 2
    assert torch.allclose(out.cpu().float(), ref, rtol=1e-2, atol=0)
    if operand:
        assert torch.equal(operand_rows(out._rb_swz, T), out)


# heads, kv heads, dim, vdim, rotated
SIZES = [(4, 4, 64, 64, 16), (6, 2, 20, 28, 12), (1, 1, 5, 2, 2),
         (8, 1, 128, 64, 32), (3, 3, 96, 128, 96), (5, 5, 64, 40, 0),
         (2, 1, 256, 192, 256), (4, 2, 72, 256, 48), (16, 2, 128, 128, 64),
         (2, 1, 300, 20, 20)]                        # the last: scalar only


@pytest.mark.parametrize("batch", list(BATCHES))
@pytest.mark.parametrize("chunk", [None, 70, 33, 1, 640])
@pytest.mark.parametrize("dtype", [BF, F32])
@pytest.mark.parametrize("size", SIZES)
def test_attention_ops_match_plain_form(size, dtype, chunk, batch):
    H, G, dim, vd, rot = size
    lay = QK.QKVLayout(H, G, dim, vd, rot)
    g = torch.Generator().manual_seed(7)
    D = 64
    r = lambda n: torch.randn(n, D, generator=g) * 2 / D ** 0.5  # noqa: E731
    w = QK.pack_qkv(lay, r(H * dim), r(G * dim), r(G * vd))
    # a query may not see what its sequence gave back
    ps = [p for p in portions(*BATCHES[batch])
          if chunk is None or p.start - p.start % chunk >= p.dropped]
    T = sum(len(p.tokens) for p in ps)
    n_y = -(-lay.n_y // 32) * 32
    y = torch.randn(T, D, generator=g) @ w.T
    y = torch.nn.functional.pad(y, (0, n_y - lay.n_y)).to(dtype)
    cos, sin = ops.rope_tables(rot, 2048, 10000.0)
    norms = torch.rand(2, dim, generator=g) + 0.5
    sink = torch.randn(H, generator=g) * 2
    cache = SK.alloc_shared_kv_cache(300, lay, "cpu", dtype)
    real = torch.zeros(lay.ec, dtype=torch.bool)     # the padding stays zero
    real[:dim] = True
    real[lay.voff:lay.voff + vd] = True
    cache.copy_((torch.randn(cache.shape, generator=g) * real).to(dtype))
    expand = SK.shared_kv_flash_supported(lay, dtype)
    n_z = -(-lay.n_z // 32) * 32
    kw = dict(chunk=chunk, out_scale=0.6)
    res = {}
    for dev in ("cpu", DEV):
        b = StepPlan(ps).build(16, [], dev, expand=expand)
        yy, cc = y.to(dev).clone(), cache.to(dev).clone()
        z = torch.zeros(T, n_z, device=dev, dtype=dtype)
        swz = None
        if dev == DEV and T <= 32 and dtype == BF:
            swz = ops.decode_operand(T, n_z, z).zero_()
        QK.qkv_prep(yy, lay, cos.to(dev), sin.to(dev), b.positions, b.slots,
                    cc, norms.to(dev), 1e-5)
        kw["sink"] = sink.to(dev)
        SK.shared_kv_attend(yy, lay, cc, b, dim ** -0.5, None, z, swz, **kw)
        if b.n_seqs > b.n_short:
            SK.shared_kv_flash(yy, lay, cc, b, dim ** -0.5, None, z, **kw)
        if swz is not None:
            assert torch.equal(operand_rows(swz, T), z)
        res[dev] = {"y": yy, "cache": cc, "z": z}
    tol = 2e-2 if dtype == BF else 3e-5
    for k in res["cpu"]:
        assert relative(res[DEV][k], res["cpu"][k]) < tol, k


@pytest.mark.parametrize("sink", [-30.0, 0.0, 7.0])
@pytest.mark.parametrize("nsplit", [1, 2, 7, 32])
def test_the_sink_counts_once_in_any_split(nsplit, sink, monkeypatch):
    lay = QK.QKVLayout(4, 2, 64, 32, 16)
    g = torch.Generator().manual_seed(1)
    ps = portions((1, 1600, 0), (5, 3, 0), (1, 0, 0), (20, 1000, 0))
    T = sum(len(p.tokens) for p in ps)
    y = torch.randn(T, 512, generator=g).to(BF)
    cache = torch.randn(300, 2, 16, lay.ec, generator=g).to(BF)
    monkeypatch.setattr(SK, "attend_split", lambda *_: nsplit)
    for chunk in (None, 300):
        res = []
        for dev in ("cpu", DEV):
            b = StepPlan(ps).build(16, [], dev)
            z = torch.zeros(T, lay.n_z, device=dev, dtype=BF)
            SK.shared_kv_attend(y.to(dev), lay, cache.to(dev), b, 0.1, None,
                                z, chunk=chunk,
                                sink=torch.full((4,), sink, device=dev))
            res.append(z)
        assert relative(res[1], res[0]) < 2e-2


@pytest.mark.parametrize("inside", [True, False])
@pytest.mark.parametrize("edge", [1, 3, 7])
@pytest.mark.parametrize("chunk", [16, 17, 31, 64])
@pytest.mark.parametrize("form", ["short", "long"])
def test_standout_key_at_the_edge_of_a_chunk(chunk, edge, inside, form):
    """A key that would take the whole output is the first of the query's
    chunk or the last of the one before: its value must fill the output or
    have no part."""
    H, G, dim, vd = 4, 2, 32, 24
    lay = QK.QKVLayout(H, G, dim, vd, 8)
    g = torch.Generator().manual_seed(edge)
    query = edge * chunk + chunk // 2
    key = edge * chunk - (0 if inside else 1)
    n = 1 if form == "short" else min(max(33, chunk), query + 1)
    if form == "long" and n <= 32:
        pytest.skip("too few tokens before the query")
    dropped = (query + 1 - n) // chunk * chunk // 16 * 16
    p = portions((n, query + 1 - n, min(dropped, key // 16 * 16)),
                 blocks=60)[0]
    cache = torch.randn(60, G, 16, lay.ec, generator=g).to(BF)
    cache[..., dim - 1] = 0
    at = key - p.dropped
    cache[p.blocks[at // 16], :, at % 16, dim - 1] = 16.0
    y = torch.zeros(n, 256, dtype=BF)
    y[:, :lay.off_k].view(n, H, dim)[..., dim - 1] = 8.0
    b = StepPlan([p]).build(16, [], DEV)
    z = torch.zeros(n, lay.n_z, dtype=BF, device=DEV)
    fn = SK.shared_kv_attend if form == "short" else SK.shared_kv_flash
    fn(y.to(DEV), lay, cache.to(DEV), b, 1.0, None, z, chunk=chunk,
       sink=torch.full((H,), -40.0, device=DEV))
    got = z[-1].float().cpu().view(H, vd)
    rows = cache[p.blocks, :, :, dim:].float().transpose(1, 2).reshape(
        -1, G, vd)                                   # values by position
    of = [h // 2 for h in range(H)]
    standout = rows[at][of]
    if inside:
        assert torch.allclose(got, standout, atol=2e-2)
    else:
        lo = edge * chunk - p.dropped
        mean = rows[lo:query + 1 - p.dropped].mean(0)[of]
        assert torch.allclose(got, mean, atol=2e-2)
        assert (got - standout).abs().max() > 0.5


# heads, q/k heads, dim, vdim, taps, ranks
STATES = [(4, 2, 64, 40, 4, 24, 16), (3, 3, 20, 12, 3, 6, 10),
          (1, 1, 1, 5, 1, 1, 1), (2, 2, 128, 128, 4, 32, 32),
          (2, 1, 256, 72, 2, 8, 40), (6, 3, 33, 200, 5, 30, 7),
          (40, 8, 16, 16, 4, 16, 16), (2, 1, 96, 264, 4, 9, 9)]


def delta_case(size, T, dtype, seed=7, decay=-1.0):
    H, G, dim, vd, taps, ra, rg = size
    lay = DR.DeltaLayout(H, G, dim, vd, taps, ra, rg)
    g = torch.Generator().manual_seed(seed)
    D = 64
    r = lambda n, k=D: torch.randn(n, k, generator=g) / k ** 0.5  # noqa: E731
    w = DR.pack_in(lay, 3 * r(G * dim), 3 * r(G * dim), 3 * r(H * vd),
                   2 * r(H), r(ra), r(rg))
    y = (torch.randn(T, D, generator=g) @ w.T).to(dtype)
    second = DR.pack_second(lay, r(H * dim, ra) * 3, r(H * vd, rg) * 2)
    y2 = (y[:, lay.off_r:lay.n_y].float() @ second.T).to(dtype)
    conv = DR.pack_conv(lay, *(0.3 + 0.5 * torch.randn(n, taps, generator=g)
                               for n in (G * dim, G * dim, H * vd)))
    dec = DR.pack_decay(lay, decay + torch.randn(H, generator=g),
                        -1 + torch.randn(H * dim, generator=g))
    return lay, y, y2, conv, dec


def delta_run(lay, y, y2, conv, dec, state, ps, dev, dtype):
    b = StepPlan(ps).build(16, [], dev,
                           expand=DR.delta_chunk_supported(lay, dtype))
    y, y2 = y.to(dev), y2.to(dev)
    o = torch.full((len(y), lay.n_o), float("nan"), device=dev)
    args = (y, y2, lay, conv.to(dev), dec.to(dev), state, b, o)
    if b.n_short:
        DR.delta_step(*args)
    if b.n_seqs > b.n_short:
        DR.delta_chunk(*args)
    n_z = -(-lay.n_o // 32) * 32
    z = torch.full((len(y), n_z), float("nan"), device=dev, dtype=dtype)
    swz = None
    if dev != "cpu" and len(y) <= 32 and dtype == BF:
        swz = ops.decode_operand(len(y), n_z, z)
    w = torch.zeros(lay.vc, device=dev)
    w[:lay.vdim] = torch.linspace(0.5, 1.5, lay.vdim, device=dev)
    DR.delta_out(o, lay, w, y2, z, 1e-5, swz, y, state[1], b)
    if swz is not None:
        assert torch.equal(operand_rows(swz, len(y)), z)
    return o, z


@pytest.mark.parametrize("batch", list(BATCHES))
@pytest.mark.parametrize("dtype", [BF, F32])
@pytest.mark.parametrize("decay", [-1.0, 3.0])       # slow, and very fast
@pytest.mark.parametrize("size", STATES)
def test_delta_rule_matches_plain_form(size, decay, dtype, batch):
    ps = portions(*BATCHES[batch])
    T = sum(len(p.tokens) for p in ps)
    lay, y, y2, conv, dec = delta_case(size, T, dtype, decay=decay)
    g = torch.Generator().manual_seed(1)
    state = DR.alloc_delta_state(len(ps), lay, "cpu", dtype)
    state[0][:, :, :lay.dim, :lay.vdim] = torch.randn(
        len(ps), lay.heads, lay.dim, lay.vdim, generator=g)
    state[1].copy_(torch.randn(state[1].shape, generator=g))
    res = {}
    for dev in ("cpu", DEV):
        st = tuple(s.to(dev).clone() for s in state)
        o, z = delta_run(lay, y, y2, conv, dec, st, ps, dev, dtype)
        res[dev] = {"o": o, "z": z, "state": st[0], "tails": st[1]}
    assert torch.equal(res[DEV]["tails"].cpu(), res["cpu"]["tails"])
    for k in ("o", "state"):
        # the recurrence keeps fp32's quality
        assert relative(res[DEV][k], res["cpu"][k]) < 1e-3, k
    assert relative(res[DEV]["z"], res["cpu"]["z"]) < (
        2e-2 if dtype == BF else 1e-3)


@pytest.mark.parametrize("size", [(4, 2, 64, 48, 4, 24, 16),
                                  (2, 1, 128, 128, 3, 16, 8)])
def test_delta_chunks_and_steps_agree(size):
    """The same tokens one by one, and through chunks at any cut of the
    portions: the same results and the same state, in fp32 quality."""
    N = 900
    lay, y, y2, conv, dec = delta_case(size, N, BF)
    out = []
    for cuts in ([1], [N], [64, 63, 300], [257, 40], [33, 2, 1, 500]):
        st = DR.alloc_delta_state(3, lay, DEV, BF)
        st[0].fill_(9.0)
        st[1].fill_(9.0)
        o = torch.zeros(N, lay.n_o, device=DEV)
        at, i = 0, 0
        while at < N:
            n = min(cuts[i % len(cuts)], N - at)
            p = portions((n, at, 0))
            p[0].slot = 1
            o[at:at + n] = delta_run(lay, y[at:at + n].contiguous(),
                                     y2[at:at + n].contiguous(), conv, dec,
                                     st, p, DEV, BF)[0]
            at, i = at + n, i + 1
        for s in st:
            assert (s[0] == 9).all() and (s[2] == 9).all()
        out.append((o, st[0][1], st[1][1].float()))
    for got in out[1:]:
        for a, ref in zip(got, out[0]):
            assert relative(a, ref.cpu()) < 2e-4


def test_delta_chunks_of_long_portions():
    """More chunks than the scratch memory holds at once, of two sequences,
    against the steps."""
    ps = portions((5000, 0, 0), (700, 300, 0), blocks=400)
    T = 5700
    lay, y, y2, conv, dec = delta_case((32, 4, 128, 128, 4, 16, 16), T, BF)
    res = []
    for expand in (True, False):
        b = StepPlan(ps).build(16, [], DEV, expand=expand)
        assert b.n_short == (0 if expand else 2)
        st = DR.alloc_delta_state(2, lay, DEV, BF)
        for x in st:
            x.fill_(0.5)
        o = torch.full((T, lay.n_o), float("nan"), device=DEV)
        run = DR.delta_chunk if expand else DR.delta_step
        run(y.to(DEV), y2.to(DEV), lay, conv.to(DEV), dec.to(DEV), st, b, o)
        res.append((o, st[0]))
    for a, ref in zip(*res):
        assert relative(a, ref.cpu()) < 1e-3


@pytest.mark.parametrize("batch", list(BATCHES) + ["long"])
@pytest.mark.parametrize("dtype", [BF, F32])
@pytest.mark.parametrize("R", [8, 40, 200, 1024])
def test_min_gru_matches_plain_form(R, dtype, batch):
    ps = portions(*{**BATCHES, "long": [(2500, 0, 0), (60, 40, 0),
                                        (1, 9, 0)]}[batch])
    T = sum(len(p.tokens) for p in ps)
    g = torch.Generator().manual_seed(2)
    y = (torch.randn(T, 3 * R + 16, generator=g) * 2).to(dtype)
    bias = torch.randn(2, R, generator=g) - 1
    state = torch.randn(len(ps), R, generator=g) * 2
    res = {}
    for dev in ("cpu", DEV):
        b = StepPlan(ps).build(16, [], dev)
        st, z = state.to(dev).clone(), torch.zeros(T, R + 8, dtype=dtype,
                                                   device=dev)
        swz = None
        if dev == DEV and T <= 32 and dtype == BF and (R + 8) % 16 == 0:
            swz = ops.decode_operand(T, R + 8, z).zero_()
        MG.min_gru(y.to(dev), 16, bias.to(dev), st, b, z, 8, 0.7, swz)
        if swz is not None:
            assert torch.equal(operand_rows(swz, T), z)
        res[dev] = (st, z)
    assert relative(res[DEV][0], res["cpu"][0]) < 1e-5
    assert relative(res[DEV][1], res["cpu"][1]) < (1e-2 if dtype == BF
                                                   else 1e-5)


# experts, top, groups, kept groups
ROUTERS = [(16, 4, 4, 3), (12, 3, 4, 2), (1, 1, 1, 1), (64, 8, 8, 1),
           (100, 5, 10, 9), (256, 8, 8, 4), (1000, 12, 1, 1), (6, 6, 2, 2)]


@pytest.mark.parametrize("T", [1, 30, 700])
@pytest.mark.parametrize("router", ROUTERS)
def test_routing(router, T):
    E, top, groups, keep = router
    g = torch.Generator().manual_seed(E)
    parts = torch.randn(2, T, E + 5, generator=g)
    bias = torch.randn(E, generator=g) * 0.2 - 0.3   # choices below zero
    ref = ME.moe_route(parts, bias, top, groups, keep)
    got = ME.moe_route(parts.to(DEV), bias.to(DEV), top, groups, keep)
    assert torch.equal(got.chosen.cpu(), ref.chosen)
    assert torch.allclose(got.weights.cpu(), ref.weights, rtol=1e-5,
                          atol=1e-8)
    for tile in (16, 128):
        pairs, tiles = ops.ext().moe_plan(got.chosen, E, tile)
        pairs, tiles = pairs.cpu(), tiles.cpu()
        assert sorted(pairs.tolist()) == list(range(T * top))
        used, seen = int(tiles[-1, 0]), 0
        assert (tiles[:, 2] > 0).sum() == used < len(tiles)
        for e, first, n, *_ in tiles.tolist():
            if n:
                assert first == seen and n <= tile
                assert (ref.chosen.view(-1)[pairs[first:first + n].long()]
                        == e).all()
                seen += n
        assert seen == T * top


# experts, top, width, inner size
EXPERTS = [(16, 4, 64, 96), (8, 2, 96, 32), (3, 3, 100, 160), (4, 1, 256, 64),
           (5, 2, 320, 288)]


@pytest.mark.parametrize("T", [1, 30, 700])
@pytest.mark.parametrize("dtype", [BF, F32])
@pytest.mark.parametrize("size", EXPERTS)
def test_expert_products(size, dtype, T):
    E, top, D, F = size
    Dp = -(-D // 32) * 32
    g = torch.Generator().manual_seed(E)
    r = lambda *n: torch.randn(*n, generator=g)  # noqa: E731
    h, up, down = r(T, Dp), r(E, F, Dp) / D ** 0.5, r(E, D, F) / F ** 0.5
    h[:, D:] = 0
    h, up, down = (t.to(dtype) for t in (h, up, down))
    logits = r(T, E)
    logits[:, 0] += 1                                # unequal loads
    res = []
    for dev in ("cpu", DEV):
        plan = ME.moe_route(logits.to(dev), torch.zeros(E, device=dev), top,
                            1, 1)
        plan = ME.moe_plan(plan, E, dtype == BF)
        a = ME.moe_up(h.to(dev), up.to(dev), plan)
        res.append((a, ME.moe_down(a, down.to(dev), plan)))
    if dtype == BF and T == 700:
        assert plan.tile == 128
    tol = 1e-2 if dtype == BF else 1e-5
    for a, ref in zip(res[1], res[0]):
        assert a.shape == ref.shape and relative(a, ref) < tol


@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("name", list(MODELS))
@pytest.mark.parametrize("cuts", [[1000], [1], [3, 40, 2, 1, 100, 17]])
def test_any_cut_of_the_prompt(name, cuts, dtype):
    cfg, W = make(name)
    toks = tokens_of(cfg, 60 if cuts == [1] else 200)
    ref = oracle.forward(cfg, W, toks)
    eng = make_engine(cfg, W, dtype, DEV)
    assert close(run_cut(eng, toks, cuts), ref, dtype, slack=1.5)
    assert len(eng.allocator.free) == eng.allocator.num_blocks
    assert len(eng.free_slots) == eng.max_batch


@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("name", ["mixed", "full"])
def test_unequal_requests_in_one_batch(name, dtype):
    """Portions beside single tokens on a small pool, pages and slots used
    again: each request's logits as if it were alone."""
    cfg, W = make(name)
    lens = [150, 3, 61, 97, 40]
    seqs = [tokens_of(cfg, n, seed=i) for i, n in enumerate(lens)]
    refs = [oracle.forward(cfg, W, s) for s in seqs]
    eng = make_engine(cfg, W, dtype, DEV, kv_blocks=20, max_batch=2)
    live, waiting, turn = {}, list(range(len(seqs))), 0
    got = [[] for _ in seqs]
    while waiting or live:
        while waiting and len(live) < 2:
            live[waiting.pop(0)] = [eng.open_request(), 0]
        entries, ids = [], []
        for i, (r, at) in live.items():
            n = min([1, 64, 2, 33, 1, 1, 5][(turn + i) % 7],
                    len(seqs[i]) - at)
            entries.append((r, seqs[i][at:at + n], range(n)))
            ids.append((i, at, n))
        turn += 1
        logits, row = eng.run_portions(entries).float().cpu(), 0
        for i, at, n in ids:
            got[i].append(logits[row:row + n])
            row += n
            live[i][1] = at + n
            if at + n == len(seqs[i]):
                eng.close_request(live.pop(i)[0])
    assert close(torch.cat([x for g in got for x in g]), torch.cat(refs),
                 dtype, slack=1.5)
    assert len(eng.allocator.free) == eng.allocator.num_blocks


def test_captured_decode_matches_eager():
    """Steps of single tokens replay a graph; between replays the engine
    runs eager steps. Same logits as without graphs."""
    cfg, W = make("mixed")
    seqs = [tokens_of(cfg, 80, seed=s) for s in range(3)]
    out = {}
    for graphs in (True, False):
        eng = make_engine(cfg, W, BF, DEV, max_batch=4)
        eng.use_graphs = graphs
        reqs = [eng.open_request() for _ in seqs]
        rows = [eng.run_portions([(r, s[:20 + 9 * i], [19 + 9 * i])])
                .float().cpu()
                for i, (r, s) in enumerate(zip(reqs, seqs))]
        at = [20, 29, 38]
        for step in range(24):
            who = [0, 1, 2] if step % 3 else [step % 2, 2]
            if step == 11:                # an eager portion in between
                rows.append(eng.run_portions(
                    [(reqs[1], seqs[1][at[1]:at[1] + 4], [3])]).float().cpu())
                at[1] += 4
            rows.append(eng.run_portions(
                [(reqs[i], seqs[i][at[i]:at[i] + 1], [0])
                 for i in who]).float().cpu().clone())
            for i in who:
                at[i] += 1
        assert (eng._graphed is not None) == graphs
        out[graphs] = torch.cat(rows)
    assert rel_err(out[True], out[False]) < 2e-2


@pytest.mark.parametrize("dtype", [F32, BF])
def test_greedy_generation_through_the_scheduler(dtype):
    """Prompts read in portions beside decoding requests. In 32-bit the
    continuation is the oracle's; in bf16 every chosen token is within
    rounding of the oracle's best."""
    cfg, W = make("mixed")
    eng = make_engine(cfg, W, dtype, DEV, max_batch=4)
    eng.prefill_chunk = 64
    prompts = [tokens_of(cfg, n, seed=n) for n in (5, 150, 33, 80, 64)]
    reqs = [eng.submit(p, max_new_tokens=40) for p in prompts]
    while eng.has_work():
        eng.step()
    for r, p in zip(reqs, prompts):
        ids = p + r.output_ids
        assert len(r.output_ids) == 40
        ref = oracle.forward(cfg, W, ids)[len(p) - 1:-1]
        if dtype == F32:
            assert ref.argmax(-1).tolist() == r.output_ids
        picked = ref.gather(1, torch.tensor(r.output_ids)[:, None])[:, 0]
        gap = ref.max(-1).values - picked
        assert float(gap.max()) < 0.3 * float(ref.std())


def test_decode_operands():
    """A width the decode GEMM takes: split slabs and pre-swizzled operands
    agree with the oracle."""
    layers = [oracle.twin(16, 4, 64, 64, 50, 16, 512, mlp=oracle.dense(1024)),
              oracle.delta(8, 4, 64, 128,
                           mlp=oracle.moe(256, 32, 4, (4, 2), 512))]
    cfg = oracle.make_config(layers, 1024, 256, 4)
    W = oracle.make_weights(cfg, 3, gain=0.7, ranks=(64, 32))
    toks = tokens_of(cfg, 60)
    ref = oracle.forward(cfg, W, toks)
    eng = make_engine(cfg, W, BF, DEV)
    for blk in eng.model.blocks:
        assert all(ops.decode_ready(w, 8) for w in (
            blk.join1.in_w, blk.mixer.out_w, blk.join2.in_w))
    assert close(run_cut(eng, toks, [40, 1, 1, 5, 1]), ref, BF)


def test_replay_command(tmp_path, monkeypatch, capsys):
    from runbooks_amd.serve.replay import main
    cfg, W = make("full")
    d = write_checkpoint(tmp_path / "m", cfg, W)
    toks = tokens_of(cfg, 70)
    ref = oracle.forward(cfg, W, toks)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": toks[:60],
                                      "want": [59]}], "end": []}] + [
        {"step": i, "entries": [{"id": "a", "tokens": [toks[59 + i]],
                                 "want": [0]}], "end": []}
        for i in range(1, 11)]
    for dtype in ("bfloat16", "float32"):
        out = tmp_path / dtype
        out.mkdir()
        monkeypatch.setattr("sys.stdin", io.StringIO(
            "".join(json.dumps(s) + "\n" for s in steps)))
        assert main(["--model", str(d), "--dtype", dtype, "--out", str(out),
                     "--max-tokens", "128"]) == 0
        got = torch.cat([torch.from_numpy(np.fromfile(
            out / f"{i}.f32", dtype="<f4")).view(1, -1) for i in range(11)])
        assert close(got, ref[59:], getattr(torch, dtype), slack=3)


def test_kernels_refuse_what_they_do_not_cover():
    """Operand errors are host-side checks, raised before any launch."""
    cfg, W = make("mixed")
    model = load(cfg, W, BF, DEV)
    idx = torch.zeros(3, dtype=torch.int32, device=DEV)
    lay = model.blocks[1].mixer.lay
    y = torch.zeros(4, 512, dtype=BF, device=DEV)
    cos, sin = (t.to(DEV) for t in ops.rope_tables(12, 16))
    cache = model.alloc_caches(2, DEV)[1][0]
    with pytest.raises(RuntimeError, match="qkv_prep"):
        QK.qkv_prep(y, lay, cos, sin, idx, idx, cache,
                    torch.ones(2, 20, device=DEV), 1e-5)
    with pytest.raises(RuntimeError, match="moe_route"):
        ME.moe_route(torch.zeros(3, 8, device=DEV),
                     torch.zeros(8, device=DEV), 5, 4, 2)
    with pytest.raises(RuntimeError, match="streams_norm"):
        ops.streams_norm(torch.zeros(2, 3, 8, device=DEV), None,
                         torch.zeros(2, device=DEV),
                         torch.zeros(17, device=DEV), BF)
    big = oracle.make_config([oracle.delta(1, 1, 300, 8)], 16, 20)
    with pytest.raises(NotImplementedError, match="no kernel"):
        make_engine(big, oracle.make_weights(big), BF, DEV)
