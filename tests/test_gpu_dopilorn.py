"""The Dopilorn family on the gfx950 kernels: each op against its plain fp32
form, whole models against the oracle, in bf16 and in 32-bit."""
import io
import json

import numpy as np
import pytest
import torch

import dopilorn_oracle as oracle
from dopilorn_helpers import (MODELS, close, load, make, make_engine,
                              portions, rel_err, run_cut, tokens_of,
                              write_checkpoint)
from runbooks_amd import ops
from runbooks_amd.models.ragged import StepPlan
from runbooks_amd.ops import canon as CA
from runbooks_amd.ops import delta as DR
from runbooks_amd.ops import general_delta as GD
from runbooks_amd.ops import latent as L
from runbooks_amd.ops import poly_norm as PN
from runbooks_amd.ops import qkv as QK
from runbooks_amd.ops import shared_kv as SK

pytestmark = pytest.mark.gpu

DEV = "cuda:0"
BF, F32 = torch.bfloat16, torch.float32
BATCHES = {"single": [(1, 0, 0), (1, 100, 0), (1, 15, 0), (1, 2, 0),
                      (1, 1500, 0)],
           "short": [(1, 0, 0), (1, 100, 0), (3, 0, 0), (2, 300, 16),
                     (1, 1500, 0), (7, 33, 0), (2, 1, 0)],
           "mixed": [(1, 640, 0), (100, 0, 0), (3, 70, 0), (33, 90, 16),
                     (200, 500, 0), (700, 0, 0), (40, 2, 0)]}


def operand_rows(swz, T):
    """Rows of a decode-GEMM operand."""
    return swz.view(-1, 2, 32, 8).permute(2, 0, 1, 3).reshape(32, -1)[:T]


def relative(a, ref):
    a, ref = a.float().cpu(), ref.float()
    if not ref.numel():
        return 0.0
    return float((a - ref).abs().max() / ref.abs().max().clamp(min=1e-20))


def randn(seed=0):
    g = torch.Generator().manual_seed(seed)
    return lambda *n: torch.randn(*n, generator=g)


def tokens_in(ps):
    return sum(len(p.tokens) for p in ps)


# --- norm and input convolution ------------------------------------------------

@pytest.mark.parametrize("batch", list(BATCHES))
@pytest.mark.parametrize("subs", [1, 2])
@pytest.mark.parametrize("D,taps", [(64, 4), (200, 1), (90, 3), (33, 7),
                                    (1024, 4), (2560, 2)])
@pytest.mark.parametrize("dtype", [BF, F32])
def test_norm_and_input_convolutions(D, taps, dtype, subs, batch):
    ps = portions(*BATCHES[batch])
    T, r = tokens_in(ps), randn(D)
    x, tails = r(T, D) * 3, r(len(ps) + 1, taps - 1, D)
    coef = CA.pack_coefficients([1 + 0.3 * r(D) for _ in range(subs)],
                                [r(D, taps) for _ in range(subs)])
    operand = dtype == BF and T <= 32
    for delta in (None, r(T, D), r(3, T, D), r(T, D).to(dtype)):
        res = {}
        for dev in ("cpu", DEV):
            xx, tt = x.to(dev).clone(), tails.to(dev).clone()
            b = StepPlan(ps).build(16, [], dev)
            hs = CA.canon_norm(xx, None if delta is None else delta.to(dev),
                               coef.to(dev), tt, b, 1e-5, dtype,
                               [operand and dev == DEV] * subs)
            res[dev] = [xx, tt, *hs]
            for h in hs:
                assert h.dtype == dtype and h.shape == (T, -(-D // 32) * 32)
                if operand and dev == DEV:
                    assert torch.equal(operand_rows(h._rb_swz, T), h)
        for i, (a, ref) in enumerate(zip(res[DEV], res["cpu"])):
            assert relative(a, ref) < (1e-5 if i < 2 or dtype == F32
                                       else 1e-2), i
        # a slot that no sequence has stays as it was
        assert torch.equal(res[DEV][1][len(ps)].cpu(), tails[len(ps)])


# heads, kv heads, dim, vdim
SIZES = [(4, 4, 64, 64), (6, 2, 20, 28), (1, 1, 5, 2), (8, 1, 64, 128),
         (3, 3, 96, 96), (5, 5, 128, 40), (2, 1, 128, 256), (6, 2, 48, 88),
         (16, 2, 16, 32), (2, 1, 256, 72), (1, 1, 256, 256), (2, 2, 10, 200),
         (3, 1, 300, 20), (2, 1, 40, 260)]         # the last two: scalar only


@pytest.mark.parametrize("batch", list(BATCHES))
@pytest.mark.parametrize("taps", [1, 3, 5])
@pytest.mark.parametrize("dtype", [BF, F32])
@pytest.mark.parametrize("size", SIZES[:5])
def test_convolution_of_queries_keys_and_values(size, taps, dtype, batch):
    lay = QK.QKVLayout(*size, maps=2)
    ps = portions(*BATCHES[batch])
    T, r = tokens_in(ps), randn(taps)
    y = torch.nn.functional.pad(r(T, lay.n_y), (0, 24)).to(dtype)
    bias, w = r(lay.n_y), r(taps, lay.n_y)
    tails = r(len(ps) + 1, taps - 1, lay.n_y).to(dtype)
    cache = SK.alloc_shared_kv_cache(300, lay, "cpu", dtype)
    res = {}
    for dev in ("cpu", DEV):
        b = StepPlan(ps).build(16, [], dev)
        tt, cc = tails.to(dev).clone(), cache.to(dev).clone()
        q = QK.qkv_conv(y.to(dev), lay, bias.to(dev), w.to(dev), tt, b, cc)
        res[dev] = (q, cc, tt)
    for a, ref in zip(res[DEV][:2], res["cpu"][:2]):
        assert relative(a, ref) < (1e-2 if dtype == BF else 1e-5)
    assert torch.equal(res[DEV][2].cpu(), res["cpu"][2])


# --- differential attention ----------------------------------------------------

def diff_case(size, dtype, ps, seed=7):
    lay, r = QK.QKVLayout(*size, maps=2), randn(seed)
    H, G, dim, vd = size
    T = tokens_in(ps)
    pad = torch.nn.functional.pad
    q = pad(r(T, 2 * H, dim) * 1.5, (0, lay.hc - dim)).view(T, -1).to(dtype)
    cache = SK.alloc_shared_kv_cache(300, lay, "cpu", dtype)
    real = torch.cat([torch.arange(lay.hc) < dim] * 2 +
                     [torch.arange(lay.vc) < vd])
    cache.copy_((r(*cache.shape) * real).to(dtype))
    return lay, q, cache


@pytest.mark.parametrize("batch", list(BATCHES))
@pytest.mark.parametrize("window", [None, 70, 33, 1, 640])
@pytest.mark.parametrize("dtype", [BF, F32])
@pytest.mark.parametrize("size", SIZES)
def test_differential_attention_matches_plain_form(size, dtype, window,
                                                   batch):
    # a query may not see what its sequence gave back
    ps = [p for p in portions(*BATCHES[batch])
          if window is None or p.start - window + 1 >= p.dropped]
    lay, q, cache = diff_case(size, dtype, ps)
    T, dim = len(q), size[2]
    expand = SK.shared_kv_flash_supported(lay, dtype)
    n_z = -(-lay.n_z // 32) * 32 + 32
    for lam in (0.4, -1.3):
        res = {}
        for dev in ("cpu", DEV):
            b = StepPlan(ps).build(16, [], dev, expand=expand)
            z = torch.zeros(T, n_z, device=dev, dtype=dtype)
            swz = None
            if dev == DEV and T <= 32 and dtype == BF:
                swz = ops.decode_operand(T, n_z, z).zero_()
            args = (q.to(dev), lay, cache.to(dev), b, dim ** -0.5, window, z)
            kw = dict(out_scale=0.6, diff=SK.DiffMaps(
                torch.tensor([lam], device=dev), lay.vdim, 1e-5))
            SK.shared_kv_attend(*args, swz, **kw)
            if b.n_seqs > b.n_short:
                SK.shared_kv_flash(*args, **kw)
            if swz is not None:
                assert torch.equal(operand_rows(swz, T), z)
            res[dev] = z
        d = (res[DEV].float().cpu() - res["cpu"].float()).abs()
        if dtype == BF:          # a difference of length near zero is noise
            assert float(d.mean()) < 3e-3 and float((d > 0.1).float().mean()
                                                    ) < 2e-3
        else:
            assert float(d.max()) < 1e-3


@pytest.mark.parametrize("nsplit", [1, 2, 7, 32])
def test_maps_meet_once_in_any_split(nsplit, monkeypatch):
    ps = portions((1, 1600, 0), (5, 3, 0), (1, 0, 0), (20, 1000, 0))
    lay, q, cache = diff_case((4, 2, 64, 96), BF, ps)
    monkeypatch.setattr(SK, "attend_split", lambda *_: nsplit)
    for window in (None, 300):
        res = []
        for dev in ("cpu", DEV):
            b = StepPlan(ps).build(16, [], dev)
            z = torch.zeros(len(q), lay.n_z, device=dev, dtype=BF)
            SK.shared_kv_attend(
                q.to(dev), lay, cache.to(dev), b, 0.1, window, z,
                diff=SK.DiffMaps(torch.tensor([0.3], device=dev), 96, 1e-5))
            res.append(z)
        assert relative(res[1], res[0]) < 2e-2


@pytest.mark.parametrize("standout_map", [0, 1])
@pytest.mark.parametrize("inside", [True, False])
@pytest.mark.parametrize("window", [1, 15, 16, 17, 31, 64, 200])
@pytest.mark.parametrize("form", ["short", "long"])
def test_standout_key_at_the_edge_of_a_window(window, inside, form,
                                              standout_map):
    """A key that would take a map's whole output is the last one inside the
    query's window, or the first one outside: its value must fill that map's
    output or have no part."""
    H, G, dim, vd = 4, 2, 32, 24
    lay = QK.QKVLayout(H, G, dim, vd, maps=2)
    g = torch.Generator().manual_seed(window)
    query = 300
    key = query - window + (1 if inside else 0)
    n = 1 if form == "short" else 70
    dropped = max(0, query - n - window) // 16 * 16
    p = portions((n, query + 1 - n, dropped), blocks=60)[0]
    cache = torch.randn(60, G, 16, lay.ec, generator=g).to(BF)
    cache[..., dim - 1] = cache[..., 2 * dim - 1] = 0
    at, col = key - p.dropped, (standout_map + 1) * dim - 1
    cache[p.blocks[at // 16], :, at % 16, col] = 16.0
    q = torch.zeros(n, 2 * H, dim, dtype=BF)
    q[..., dim - 1] = 8.0
    b = StepPlan([p]).build(16, [], DEV)
    z = torch.zeros(n, lay.n_z, dtype=BF, device=DEV)
    fn = SK.shared_kv_attend if form == "short" else SK.shared_kv_flash
    fn(q.view(n, -1).to(DEV), lay, cache.to(DEV), b, 1.0, window, z,
       diff=SK.DiffMaps(torch.tensor([0.5], device=DEV), vd, 1e-6))
    rows = cache[p.blocks, :, :, 2 * dim:].float().transpose(1, 2).reshape(
        -1, G, vd)                                   # values by position
    lo = max(0, query - window + 1) - p.dropped
    mean = rows[lo:query + 1 - p.dropped].mean(0)
    a = [mean, mean]
    if inside:
        a[standout_map] = rows[at]
    ref = oracle.rms((a[0] - 0.5 * a[1]).double(), 1e-6)
    got = z[-1].float().cpu().view(G, H // G, vd)
    assert torch.allclose(got.double(), ref[:, None].expand(got.shape),
                          atol=5e-2)


# --- latent attention without positions ------------------------------------------

# heads, dim, vdim, query rank, rank
LATENTS = [(9, 128, 128, 96, 512), (5, 12, 20, 28, 36), (1, 1, 1, 1, 1),
           (16, 64, 64, 64, 128), (3, 200, 256, 40, 72), (40, 64, 96, 33, 200),
           (2, 24, 10, 50, 64), (2, 300, 24, 8, 600)]   # the last: scalar


@pytest.mark.parametrize("batch", list(BATCHES))
@pytest.mark.parametrize("dtype", [BF, F32])
@pytest.mark.parametrize("size", LATENTS)
def test_latent_attention_matches_plain_form(size, dtype, batch):
    H, dim, vd, rq, rank = size
    lay = L.LatentLayout(H, dim, 0, vd, rank, 0, own_latent=False)
    ps, r = portions(*BATCHES[batch]), randn(3)
    T = tokens_in(ps)
    uk = r(H * dim, rank) / rank ** 0.5
    uv = r(H * vd, rank) / rank ** 0.5
    q = torch.nn.functional.pad(r(T, H, dim), (0, lay.dimc - dim)).view(T, -1)
    gate = r(T, 8 + -(-H // 8) * 8) * 2
    cache = torch.zeros(300, 16, lay.ec)
    cache[..., :rank] = r(300, 16, rank)
    q, gate, cache, uk, uv = (t.to(dtype) for t in (q, gate, cache, uk, uv))
    expand = L.latent_flash_supported(lay, dtype) and dtype == BF
    pad = torch.nn.functional.pad
    n_z = -(-lay.off_act // 32) * 32
    res = {}
    for dev in ("cpu", DEV):
        b = StepPlan(ps).build(16, [None], dev, expand=expand)
        qq, gg, cc, k, v = (t.to(dev) for t in (q, gate, cache, uk, uv))
        c = lay.rc - rank
        absorb = L.pack_heads(pad(k.view(H, dim, -1),
                                  (0, c, 0, lay.dimc - dim)))
        ex = L.pack_heads(pad(v.view(H, vd, -1), (0, c, 0, lay.vc - vd)
                              ).transpose(1, 2))
        z = torch.zeros(T, n_z, device=dev, dtype=dtype)
        swz = None
        if dev == DEV and T <= 32 and dtype == BF:
            swz = ops.decode_operand(T, n_z, z).zero_()
        if b.t_short:
            lat = L.latent_absorb(qq, lay, absorb, b.t_short)
            lat = L.latent_attend(lat, qq, lay, cc, b, dim ** -0.5, None)
            L.latent_expand(lat, lay, ex, gg, z, swz, off_g=8, head_gate=True)
        if b.long_plans:
            slots, meta = b.long_plans[None]
            ctx = cc.view(-1, lay.ec).index_select(0, slots)
            kv = torch.nn.functional.linear(ctx, L.pack_expand(lay, k, v))
            L.latent_flash(qq, lay, kv, ctx, meta, b.max_q_long, dim ** -0.5,
                           None, z, gg, off_g=8, head_gate=True)
        if swz is not None:
            assert torch.equal(operand_rows(swz, T), z)
        res[dev] = z
    assert relative(res[DEV], res["cpu"]) < (2e-2 if dtype == BF else 3e-5)


@pytest.mark.parametrize("T", [1, 32, 300])
@pytest.mark.parametrize("dtype", [BF, F32])
@pytest.mark.parametrize("rq,rank", [(64, 512), (1, 3), (1500, 24),
                                     (5000, 9000)])
def test_norms_of_both_latents(rq, rank, dtype, T):
    r, off = randn(T), 8 + -(-rq // 8) * 8
    y = r(T, off + -(-rank // 8) * 8).to(dtype)
    slots = torch.randperm(320, generator=torch.Generator().manual_seed(1))
    slots = slots[:T].int()
    wq, wc = r(rq), r(rank)
    operand = dtype == BF and T <= 32
    res = {}
    for dev in ("cpu", DEV):
        cache = torch.zeros(20, 16, -(-rank // 8) * 8, dtype=dtype,
                            device=dev)
        swz = None
        if operand and dev == DEV:
            swz = ops.decode_operand(T, -(-rq // 32) * 32, cache)
        out = L.latent_norms(y.to(dev), ((8, off), (rq, rank),
                                         (wq.to(dev), wc.to(dev))), 1e-5,
                             slots.to(dev), cache, swz)
        res[dev] = (out, cache)
        if swz is not None:
            assert torch.equal(operand_rows(out._rb_swz, T), out)
    for a, ref in zip(res[DEV], res["cpu"]):
        assert a.shape == ref.shape
        assert relative(a, ref) < (1e-2 if dtype == BF else 1e-5)


def test_standout_key_far_back_in_the_latents():
    """One key far back takes the whole output, for a decoded token and at
    every cut of a portion."""
    H, dim, rank, query = 4, 32, 64, 1400
    lay = L.LatentLayout(H, dim, 0, 16, rank, 0, own_latent=False)
    r = randn(2)
    for key in (0, 15, 16, 700, 1399, 1400):
        p = portions((1, query, 0), blocks=100)[0]
        cache = r(100, 16, lay.ec).to(BF)
        cache[..., 0] = 0
        cache[p.blocks[key // 16], key % 16, 0] = 16.0
        q_lat = torch.zeros(1, H, rank, dtype=BF)
        q_lat[..., 0] = 8.0
        b = StepPlan([p]).build(16, [None], DEV)
        y = torch.zeros(1, H * dim, dtype=BF, device=DEV)
        out = L.latent_attend(q_lat.to(DEV), y, lay, cache.to(DEV), b, 1.0,
                              None)
        want = cache[p.blocks[key // 16], key % 16]
        assert torch.equal(out.cpu(), want.expand(1, H, rank))


# --- generalized delta rule ----------------------------------------------------

# heads, dim, value columns, bottleneck
STATES = [(4, 64, 64, 24), (3, 20, 20, 6), (1, 1, 1, 1), (2, 128, 128, 32),
          (2, 256, 256, 8), (6, 33, 33, 30), (20, 16, 16, 16), (2, 96, 40, 9),
          (1, 136, 200, 5)]


def delta_case(size, T, dtype, seed=7, scale=2.0):
    H, dim, vd, rank = size
    lay, r = GD.GeneralDeltaLayout(*size), randn(seed)
    D = 64

    def lin(n, k=D):
        return r(n, k) / k ** 0.5

    w = GD.pack_in(lay, lin(H * dim), 2 * lin(H * dim), lin(H * vd),
                   scale * lin(H * dim), lin(H * vd), lin(rank))
    y = (r(T, D) @ w.T).to(dtype)
    y2 = (torch.tanh(y[:, lay.off_r:lay.n_y].float()) @ GD.pack_second(
        lay, scale * lin(H * dim, rank)).T).to(dtype)
    bias = GD.pack_bias(lay, r(H * dim), r(H * dim))
    return lay, y, y2, bias


def delta_run(lay, y, y2, bias, state, ps, dev, scale=-0.60653, expand=None):
    if expand is None:
        expand = GD.general_delta_chunk_supported(lay, y.dtype)
    b = StepPlan(ps).build(16, [], dev, expand=expand)
    o = torch.full((len(y), lay.n_o), float("nan"), device=dev)
    args = (y.to(dev), y2.to(dev), lay, bias.to(dev), scale, state, b, o)
    if b.n_short:
        GD.general_delta_step(*args)
    if b.n_seqs > b.n_short:
        GD.general_delta_chunk(*args)
    return o


@pytest.mark.parametrize("batch", list(BATCHES))
@pytest.mark.parametrize("dtype", [BF, F32])
@pytest.mark.parametrize("scale", [-0.60653, -2.0, -0.01])
@pytest.mark.parametrize("size", STATES)
def test_delta_rule_matches_plain_form(size, scale, dtype, batch):
    ps = portions(*BATCHES[batch])
    T, r = tokens_in(ps), randn(1)
    lay, y, y2, bias = delta_case(size, T, dtype)
    H, dim, vd, _ = size
    state = GD.alloc_general_delta_state(len(ps), lay, "cpu")
    state[:, :, :dim, :vd] = r(len(ps), H, dim, vd)
    res = {}
    for dev in ("cpu", DEV):
        st = state.to(dev).clone()
        res[dev] = (delta_run(lay, y, y2, bias, st, ps, dev, scale), st)
    for a, ref in zip(res[DEV], res["cpu"]):
        # the recurrence keeps fp32's quality
        assert relative(a, ref) < (3e-4 if dtype == BF else 2e-5)


@pytest.mark.parametrize("size", [(4, 64, 64, 24), (2, 128, 128, 16),
                                  (3, 40, 40, 8)])
def test_delta_chunks_and_steps_agree(size):
    """The same tokens one by one, and through chunks at any cut of the
    portions: the same results and the same state, in fp32 quality."""
    N = 900
    lay, y, y2, bias = delta_case(size, N, BF)
    out = []
    for cuts in ([1], [N], [64, 63, 300], [257, 40], [33, 2, 1, 500]):
        st = GD.alloc_general_delta_state(3, lay, DEV).fill_(9.0)
        o = torch.zeros(N, lay.n_o, device=DEV)
        at, i = 0, 0
        while at < N:
            n = min(cuts[i % len(cuts)], N - at)
            p = portions((n, at, 0))
            p[0].slot = 1
            o[at:at + n] = delta_run(lay, y[at:at + n].contiguous(),
                                     y2[at:at + n].contiguous(), bias, st, p,
                                     DEV)
            at, i = at + n, i + 1
        assert (st[0] == 9).all() and (st[2] == 9).all()
        out.append((o, st[1]))
    for got in out[1:]:
        for a, ref in zip(got, out[0]):
            assert relative(a, ref.cpu()) < 2e-4


def test_delta_chunks_of_long_portions():
    """More chunks than the scratch memory holds at once, of two sequences,
    against the steps."""
    ps = portions((5000, 0, 0), (700, 300, 0), blocks=400)
    lay, y, y2, bias = delta_case((32, 128, 128, 16), 5700, BF)
    res = []
    for expand in (True, False):
        st = GD.alloc_general_delta_state(2, lay, DEV).fill_(0.5)
        res.append((delta_run(lay, y, y2, bias, st, ps, DEV, expand=expand),
                    st))
    for a, ref in zip(*res):
        assert relative(a, ref.cpu()) < 1e-3


def test_repeated_keys_are_removed_and_written_again():
    """One key over and over with a removal rate near 1: (I + A) is as far
    from the identity as it gets."""
    N, size = 200, (2, 64, 64, 8)
    lay, y, y2, bias = delta_case(size, N, BF)
    y[:, lay.off_k:lay.off_v] = y[:1, lay.off_k:lay.off_v]
    y[:, lay.off_a:lay.off_g] = 8.0
    y2.fill_(-9.0)                                   # hardly any decay
    res = []
    for dev, dt in (("cpu", F32), (DEV, BF)):
        st = GD.alloc_general_delta_state(1, lay, dev)
        res.append(delta_run(lay, y.to(dt), y2.to(dt), bias, st,
                             portions((N, 0, 0)), dev))
    assert relative(res[1], res[0]) < 3e-4


@pytest.mark.parametrize("T", [1, 32, 40])
@pytest.mark.parametrize("dtype", [BF, F32])
@pytest.mark.parametrize("size", STATES[:7])
def test_delta_output_with_weights_of_all_heads(size, dtype, T):
    lay, y, y2, _ = delta_case(size, T, dtype)
    r = randn(4)
    o, w = r(T, lay.n_o), GD.pack_norm(lay, r(lay.heads * lay.vdim))
    pad = torch.arange(lay.n_o) % lay.vc >= lay.vdim
    o[:, pad] = 0
    end, n_z = lay.n_o, -(-lay.n_o // 32) * 32 + 32
    res = {}
    for dev in ("cpu", DEV):
        b = StepPlan(portions((T, 0, 0))).build(16, [], dev)
        z = torch.full((T, n_z), 7.0, device=dev, dtype=dtype)
        swz = None
        if dev == DEV and T <= 32 and dtype == BF:
            swz = ops.decode_operand(T, n_z, z).fill_(7.0)
        DR.delta_out(o.to(dev), lay, w.to(dev), y.to(dev), z, 1e-5, swz,
                     y.to(dev), None, b, end=end)
        if swz is not None:
            assert torch.equal(operand_rows(swz, T), z)
        res[dev] = z
    assert (res[DEV][:, end:] == 7).all()            # not its columns
    assert relative(res[DEV], res["cpu"]) < (1e-2 if dtype == BF else 1e-5)


# --- activations -----------------------------------------------------------------

@pytest.mark.parametrize("T,ff", [(1, 32), (32, 411), (33, 416), (300, 1024),
                                  (5, 16384), (2, 1)])
@pytest.mark.parametrize("dtype", [BF, F32])
def test_poly_norm(T, ff, dtype):
    r = randn(ff)
    ny = -(-ff // 32) * 32 + 32
    u, act = (r(T, ny) * 2).to(dtype), r(4)
    off, n_z = 24, -(-(24 + ff) // 32) * 32
    act[3] = 0.25
    res = {}
    for dev in ("cpu", DEV):
        for given in (False, True):
            z = torch.full((T, n_z), 7.0, device=dev, dtype=dtype)
            swz = None
            if dev == DEV and T <= 32 and dtype == BF:
                swz = ops.decode_operand(T, n_z, z).fill_(7.0)
            sums = PN.power_sums(u.to(dev), ff) if given else None
            PN.poly_norm(u.to(dev), ff, ff, act.to(dev), 1e-5, z, off, swz,
                         sums)
            if swz is not None:
                assert torch.equal(operand_rows(swz, T), z)
            res[dev, given] = z
    ref = oracle.poly_norm(u[:, :ff].double(), act.double().tolist(), 1e-5)
    z = res[DEV, False].cpu()
    assert (z[:, :off] == 7).all() and not z[:, off + ff:].any()
    assert relative(z[:, off:off + ff], ref) < (1e-2 if dtype == BF else 1e-5)
    for key, z in res.items():
        assert relative(z, res["cpu", False]) < (1e-2 if dtype == BF
                                                 else 1e-5), key


@pytest.mark.parametrize("T,n", [(1, 32), (32, 96), (33, 128)])
@pytest.mark.parametrize("dtype", [BF, F32])
def test_tanh_rows(T, n, dtype):
    y = (randn(n)(T, n + 24) * 3).to(dtype)
    operand = dtype == BF and T <= 32
    out = GD.tanh_rows(y.to(DEV), 16, n, operand)
    ref = GD.tanh_rows(y, 16, n, False)
    assert relative(out, ref) < (1e-2 if dtype == BF else 1e-6)
    if operand:
        assert torch.equal(operand_rows(out._rb_swz, T), out)


@pytest.mark.parametrize("shape", [(3, 5, 640), (1, 33), (4, 77), (1, 2, 7)])
def test_softcap(shape):
    x = randn(1)(*shape) * 40
    for cap in (5.0, 30.0):
        got, ref = ops.softcap(x.to(DEV), cap), ops.softcap(x, cap)
        assert got.shape == ref.shape and relative(got, ref) < 1e-6


# --- whole models ------------------------------------------------------------------

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
@pytest.mark.parametrize("name", ["mixed", "windows"])
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
    layers = [oracle.diff(8, 4, 64, 128, 50, mlp=oracle.dense(1024)),
              oracle.latent(8, 64, 64, 1024, 128, mlp=oracle.dense(512)),
              oracle.delta(8, 64, mlp=oracle.dense(1024))]
    cfg = oracle.make_config(layers, 1024, 256, (1, 3, 2))
    W = oracle.make_weights(cfg, 3, gain=0.7, rank=64)
    toks = tokens_of(cfg, 60)
    ref = oracle.forward(cfg, W, toks)
    eng = make_engine(cfg, W, BF, DEV)
    m = eng.model
    assert ops.decode_ready(m.loop_in.weight, 8)
    assert ops.decode_ready(m.lm_head.weight, 8)
    for blk in m.blocks:
        assert all(ops.decode_ready(w, 8) for w in (
            blk.mixer.in_w, blk.mlp.in_w, blk.out_w))
    assert ops.decode_ready(m.blocks[1].mixer.q_w, 8)
    assert close(run_cut(eng, toks, [40, 1, 1, 5, 1]), ref, BF)


def test_replay_command(tmp_path, monkeypatch, capsys):
    from runbooks_amd.serve.replay import main
    cfg, W = make("mixed")
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
    for blk in model.blocks:
        blk.fuse()
    b = StepPlan(portions((3, 0, 0))).build(16, [], DEV)
    y = torch.zeros(4, 512, dtype=BF, device=DEV)
    (cache, tails), canon = model.alloc_caches(2, DEV)[0]
    mixer = model.blocks[0].mixer
    with pytest.raises(RuntimeError, match="qkv_conv"):
        QK.qkv_conv(y, mixer.lay, mixer.bias, mixer.conv_w, tails, b, cache)
    with pytest.raises(RuntimeError, match="canon_norm"):
        CA.canon_norm(torch.zeros(3, 40, device=DEV), None,
                      model.blocks[0].coef, canon, b, 1e-5, BF, [False])
    with pytest.raises(RuntimeError, match="decay scale"):
        lay, y, y2, bias = delta_case((2, 16, 16, 4), 3, BF)
        delta_run(lay, y, y2, bias,
                  GD.alloc_general_delta_state(1, lay, DEV),
                  portions((3, 0, 0)), DEV, scale=-3.0)
    with pytest.raises(RuntimeError, match="two maps"):
        SK.shared_kv_attend(
            torch.zeros(3, mixer.lay.off_k, dtype=BF, device=DEV), mixer.lay,
            cache, b, 1.0, None,
            torch.zeros(3, mixer.lay.n_z, dtype=BF, device=DEV),
            diff=SK.DiffMaps(torch.zeros(2, device=DEV), 28, 1e-5))
    big = oracle.make_config([oracle.delta(1, 300)], 16, 20)
    with pytest.raises(NotImplementedError, match="no kernel"):
        make_engine(big, oracle.make_weights(big), BF, DEV)
