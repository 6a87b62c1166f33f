"""Latent attention on the gfx950 kernels: each op against its plain fp32
form, whole models against the oracle, in bf16 and in 32-bit."""
import io
import json

import numpy as np
import pytest
import torch

import latent_oracle as oracle
from latent_helpers import (MODELS, close, load, make, make_engine, rel_err,
                            run_cut, tokens_of, write_checkpoint)
from runbooks_amd import ops
from runbooks_amd.models.config import GatedMLPSpec
from runbooks_amd.models.ragged import Portion, StepPlan
from runbooks_amd.ops import latent as L

pytestmark = pytest.mark.gpu

DEV = "cuda:0"
BF, F32 = torch.bfloat16, torch.float32


@pytest.mark.parametrize("T,D", [(1, 64), (7, 200), (32, 256), (33, 90),
                                 (300, 1024)])
@pytest.mark.parametrize("dtype", [BF, F32])
def test_rmsnorm_res32(T, D, dtype):
    g = torch.Generator().manual_seed(0)
    x = torch.randn(T, D, generator=g)
    w = torch.rand(D, generator=g).to(dtype)
    deltas = [None, torch.randn(T, D, generator=g),
              torch.randn(T, D, generator=g).to(BF),
              torch.randn(3, T, D, generator=g)]
    for d in deltas:
        add = 0 if d is None else d.float() if d.dim() == 2 else d.sum(0)
        y = x.to(DEV)
        operand = dtype == BF and T <= 32 and D % 16 == 0
        out = ops.rmsnorm_res32(y, None if d is None else d.to(DEV),
                                w.to(DEV), 1e-3, dtype, operand=operand)
        assert torch.allclose(y.cpu(), x + add, atol=1e-5)
        ref = oracle.rms_norm((x + add).double(), w.double(), 1e-3)
        tol = 2e-2 if dtype == BF else 1e-5
        assert out.dtype == dtype
        assert torch.allclose(out.cpu().double(), ref, atol=tol, rtol=tol)
        if operand:
            rows = out._rb_swz.view(-1, 2, 32, 8).permute(2, 0, 1, 3)
            assert torch.equal(rows.reshape(32, D)[:T], out)


def _portions(spec, blocks=300, seed=2):
    g = torch.Generator().manual_seed(seed)
    free = torch.randperm(blocks, generator=g).tolist()
    out = []
    for n, start, dropped in spec:
        nb = -(-(start + n - dropped) // 16)
        out.append(Portion([0] * n, start, dropped,
                           [free.pop() for _ in range(nb)], []))
    return out


SIZES = [(4, 32, 16, 32, 64, 96), (3, 20, 12, 18, 36, 50),
         (1, 64, 8, 128, 200, 0), (5, 128, 64, 128, 512, 300),
         (16, 96, 16, 64, 128, 64), (40, 128, 64, 100, 256, 40),
         (2, 200, 40, 160, 600, 64),    # beyond the MFMA tiles
         (2, 64, 80, 64, 64, 64)]
BATCHES = {"short": [(1, 0, 0), (1, 100, 0), (1, 15, 0), (2, 300, 16),
                     (1, 1500, 0)],
           "mixed": [(1, 640, 0), (100, 0, 0), (3, 70, 0), (33, 90, 16),
                     (200, 500, 0)]}


@pytest.mark.parametrize("batch", list(BATCHES))
@pytest.mark.parametrize("window", [None, 70, 33, 1])
@pytest.mark.parametrize("dtype", [BF, F32])
@pytest.mark.parametrize("size", SIZES)
def test_ops_match_plain_form(size, dtype, window, batch):
    H, dim, rot, vd, R, F = size
    lay = L.LatentLayout(H, dim, rot, vd, R, F, True)
    g = torch.Generator().manual_seed(7)
    r = lambda *s: torch.randn(*s, generator=g) / s[-1] ** 0.5  # noqa: E731
    D, scale = 64, 0.2
    wide = L.pack_wide(lay, r(H * (dim + rot), D) * 2, r(R + rot, D) * 2,
                       r(H * vd, D), r(F, D) * 2 if F else None,
                       r(F, D) * 2 if F else None)
    uk, uv = r(H * dim, R), r(H * vd, R)
    portions = _portions(BATCHES[batch])
    T = sum(len(p.tokens) for p in portions)
    y = (torch.randn(T, D, generator=g) @ wide.T).to(dtype)
    cos, sin = ops.rope_tables(rot, 2048, 10000.0)
    cache = L.alloc_latent_cache(300, lay, "cpu", dtype)
    flat = cache.view(-1, lay.ec)
    flat[:, :R] = torch.randn(4800, R, generator=g).to(dtype)
    flat[:, lay.rc:lay.rc + rot] = torch.randn(4800, rot,
                                               generator=g).to(dtype)
    norm = torch.rand(R, generator=g).to(dtype)
    mlp = GatedMLPSpec(F, 1.2) if F else None
    pad = torch.nn.functional.pad
    wa = pad(uk.view(H, dim, R), (0, lay.rc - R, 0,
                                  lay.dimc - dim)).to(dtype)
    we = pad(uv.view(H, vd, R),
             (0, lay.rc - R, 0, lay.vc - vd)).transpose(1, 2).to(dtype)
    wc = L.pack_expand(lay, uk, uv).to(dtype)
    expand = dtype == BF and L.latent_flash_supported(lay, dtype)

    res = {}
    for dev in ("cpu", DEV):
        b = StepPlan(portions).build(16, [window], dev, expand=expand)
        yy, cc = y.to(dev).clone(), cache.to(dev).clone()
        z = torch.full((T, lay.n_z), float("nan"), device=dev, dtype=dtype)
        swz = None
        if dev == DEV and T <= 32 and dtype == BF:
            swz = ops.decode_operand(T, lay.n_z, z)
        L.latent_prep(yy, lay, cos.to(dev), sin.to(dev), b.positions,
                      b.slots, cc, norm.to(dev), 1e-5, mlp, z, swz)
        ql = L.latent_absorb(yy, lay, L.pack_heads(wa.to(dev)), b.t_short)
        ol = L.latent_attend(ql, yy, lay, cc, b, scale, window)
        L.latent_expand(ol, lay, L.pack_heads(we.to(dev)), yy, z, swz)
        if b.long_plans:
            slots, meta = b.long_plans[window]
            ctx = cc.view(-1, lay.ec).index_select(0, slots)
            kv = torch.nn.functional.linear(ctx[:, :lay.rc], wc.to(dev))
            L.latent_flash(yy, lay, kv, ctx, meta, b.max_q_long, scale,
                           window, z)
        if swz is not None:
            rows = swz.view(-1, 2, 32, 8).permute(2, 0, 1, 3)
            assert torch.equal(rows.reshape(32, -1)[:T], z)
        res[dev] = {"y": yy, "cache": cc, "q_lat": ql, "o_lat": ol, "z": z}
    tol = 2e-2 if dtype == BF else 2e-5
    for k in res["cpu"]:
        a, ref = res[DEV][k].float().cpu(), res["cpu"][k].float()
        err = (a - ref).abs().max() / ref.abs().max()
        assert err < tol, (k, float(err))


@pytest.mark.parametrize("inside", [True, False])
@pytest.mark.parametrize("query", [101, 111, 112, 127, 200, 255])
@pytest.mark.parametrize("window", [17, 64, 100])
@pytest.mark.parametrize("form", ["latent", "expanded"])
def test_standout_key_at_the_window_edge(window, query, inside, form):
    """A key that would take the whole output sits just inside or just
    outside the window: its value must fill the output or have no part."""
    H, dim, rot, vd, R = 4, 32, 16, 32, 64
    lay = L.LatentLayout(H, dim, rot, vd, R, 0, True)
    g = torch.Generator().manual_seed(query)
    cache = L.alloc_latent_cache(20, lay, "cpu", BF)
    flat = cache.view(-1, lay.ec)
    flat[:, :R] = torch.randn(320, R, generator=g).to(BF)
    key = query - window + (1 if inside else 0)
    # portion of 40 queries (200..) or of one (decoding), ending at `query`
    n = 1 if form == "latent" else min(40, query + 1)
    p = _portions([(n, query + 1 - n, 0)], blocks=20)[0]
    slot = p.blocks[key // 16] * 16 + key % 16
    flat[slot, R] = 16.0                  # rotated part: one unit apart
    y = torch.zeros(n, lay.n_y)
    y[:, :lay.off_kv].view(n, H, lay.qc)[..., lay.dimc] = 8.0
    y[:, lay.off_g:lay.off_gate] = 30.0   # open gates
    uv = torch.zeros(H, vd, R)
    for h in range(H):
        uv[h, :, h * 8:h * 8 + vd] = torch.eye(vd)
    y, cache = y.to(BF).to(DEV), cache.to(DEV)
    b = StepPlan([p]).build(16, [window], DEV, expand=form == "expanded")
    z = torch.zeros(n, lay.n_z, dtype=BF, device=DEV)
    if form == "latent":
        ql = torch.zeros(n, H, R, dtype=BF, device=DEV)
        ol = L.latent_attend(ql, y, lay, cache, b, 1.0, window)
        L.latent_expand(ol, lay, L.pack_heads(
            uv.transpose(1, 2).to(BF).to(DEV)), y, z)
    else:
        import runbooks_amd.models.ragged as ragged
        keep, ragged.ABSORB_MAX = ragged.ABSORB_MAX, 0
        try:
            b = StepPlan([p]).build(16, [window], DEV)
        finally:
            ragged.ABSORB_MAX = keep
        slots, meta = b.long_plans[window]
        ctx = cache.view(-1, lay.ec).index_select(0, slots)
        wc = L.pack_expand(lay, torch.zeros(H * dim, R),
                           uv.view(-1, R)).to(BF).to(DEV)
        L.latent_flash(y, lay, ctx[:, :R] @ wc.T, ctx, meta, b.max_q_long,
                       1.0, window, z)
    got = z[-1, :lay.off_act].float().cpu().view(H, vd)
    standout = torch.einsum("hvr,r->hv", uv, flat[slot, :R].float())
    if inside:
        assert torch.allclose(got, standout, atol=2e-2)
    else:
        pos = torch.arange(query - window + 1, query + 1)
        rows = torch.tensor([p.blocks[i // 16] * 16 + i % 16
                             for i in pos.tolist()])
        mean = torch.einsum("hvr,kr->hv", uv, flat[rows, :R].float()) / window
        assert torch.allclose(got, mean, atol=2e-2)
        assert (got - standout).abs().max() > 0.5


@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("name", list(MODELS))
@pytest.mark.parametrize("cuts", [[1000], [1], [3, 40, 2, 1, 100, 17]])
def test_any_cut_of_the_prompt(name, cuts, dtype):
    cfg, W = make(name)
    toks = tokens_of(cfg, 90 if cuts == [1] else 260)
    ref = oracle.forward(cfg, W, toks)
    eng = make_engine(cfg, W, dtype, DEV)
    assert close(run_cut(eng, toks, cuts), ref, dtype)
    assert len(eng.allocator.free) == eng.allocator.num_blocks


@pytest.mark.parametrize("dtype", [F32, BF])
def test_unequal_requests_in_one_batch(dtype):
    """Portions beside single tokens on a small pool, pages used again: each
    request's logits as if it were alone."""
    cfg, W = make("full")
    lens = [150, 3, 61, 97, 40]
    seqs = [tokens_of(cfg, n, seed=i) for i, n in enumerate(lens)]
    refs = [oracle.forward(cfg, W, s) for s in seqs]
    eng = make_engine(cfg, W, dtype, DEV, kv_blocks=20, max_batch=4)
    live, waiting, turn = {}, list(range(len(seqs))), 0
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
            assert close(logits[row:row + n], refs[i][at:at + n], dtype,
                         slack=3)
            row += n
            live[i][1] = at + n
            if at + n == len(seqs[i]):
                eng.close_request(live.pop(i)[0])
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
    eng = make_engine(cfg, W, dtype, DEV, max_batch=4, prefix_cache=True)
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


def test_decode_operands_and_8bit_weights():
    """A width the decode GEMM takes: split slabs, pre-swizzled operands and
    the fp8 weight mode run and agree with the oracle."""
    layers = [dict(heads=8, dim=32, rot_dim=16, vdim=128, kv_rank=64,
                   window=50, ff=1024, limit=2.0)] * 2
    cfg = oracle.make_config(layers, 1024, 256)
    W = oracle.make_weights(cfg, 3, gain=0.7)
    toks = tokens_of(cfg, 40)
    ref = oracle.forward(cfg, W, toks)
    eng = make_engine(cfg, W, BF, DEV)
    assert all(ops.decode_ready(w, 8) for b in eng.model.blocks
               for w in (b.wide_w, b.out_w))
    assert close(run_cut(eng, toks, [30, 1, 1, 5, 1]), ref, BF)
    e8 = make_engine(cfg, W, BF, DEV, load_in_8bit=True)
    assert rel_err(run_cut(e8, toks, [30, 1, 1, 5, 1]), ref) < 0.3


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
    lay = model.blocks[0].lay
    y = torch.zeros(4, lay.n_y, dtype=BF, device=DEV)
    z = torch.zeros(3, lay.n_z, dtype=BF, device=DEV)
    idx = torch.zeros(4, dtype=torch.int32, device=DEV)
    cos, sin = (t.to(DEV) for t in ops.rope_tables(12, 16))
    with pytest.raises(RuntimeError, match="latent_prep"):
        L.latent_prep(y, lay, cos, sin, idx, idx, model.alloc_caches(2, DEV)[0],
                      torch.ones(36, dtype=BF, device=DEV), 1e-5,
                      GatedMLPSpec(50, 1.0), z)
