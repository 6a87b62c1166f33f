"""The Dopilorn family on the CPU path: every op and whole engine runs against
the plain oracle (tests/dopilorn_oracle.py)."""
import io
import json
import os

import numpy as np
import pytest
import torch

import dopilorn_oracle as oracle
from dopilorn_helpers import (MODELS, load, make, make_engine, portions,
                              rel_err, run_cut, tokens_of, write_checkpoint)
from runbooks_amd import ops
from runbooks_amd.models import build_model, get_config
from runbooks_amd.models.config import (DiffAttentionSpec, GeneralDeltaSpec,
                                        GLUSpec, LatentAttentionSpec,
                                        LayerSpec, LoopSpec, PolyNormSpec,
                                        layered_config)
from runbooks_amd.models.load import (config_from_dir, config_from_dopilorn,
                                      config_to_dopilorn, load_pretrained)
from runbooks_amd.models.ragged import StepPlan
from runbooks_amd.ops import canon as CA
from runbooks_amd.ops import delta as DR
from runbooks_amd.ops import general_delta as GD
from runbooks_amd.ops import latent as L
from runbooks_amd.ops import poly_norm as PN
from runbooks_amd.ops import qkv as QK
from runbooks_amd.ops import shared_kv as SK
from runbooks_amd.serve import Engine

TOL = 3e-5


def shapes_of(W):
    return {k: tuple(v.shape) for k, v in W.items()}


def randn(seed=0):
    g = torch.Generator().manual_seed(seed)
    return lambda *n: torch.randn(*n, generator=g)


def cut_portions(T, cuts, blocks):
    """One sequence in portions of the given sizes, on one slot and set of
    pages."""
    out, at, i = [], 0, 0
    pages = portions((T, 0, 0), blocks=blocks)[0].blocks
    while at < T:
        n = min(cuts[i % len(cuts)], T - at)
        p = portions((n, at, 0), blocks=blocks)[0]
        p.blocks, p.slot = pages[:-(-(at + n) // 16)], 1
        out.append((at, n, p))
        at, i = at + n, i + 1
    return out


CUTS = [[1], [1000], [2, 5, 1, 40]]


# --- single mechanisms -------------------------------------------------------

@pytest.mark.parametrize("cuts", CUTS)
@pytest.mark.parametrize("taps", [1, 2, 4, 9])
def test_norm_and_input_convolution(taps, cuts):
    """Norm, convolution and residual sum at any cut; two sublayers share
    the normed rows."""
    T, D, r = 70, 20, randn(taps)
    x, w, c = r(T, D) * 3, [r(D), r(D)], [r(D, taps), r(D, taps)]
    delta = r(3, T, D)
    coef = CA.pack_coefficients([1 + v for v in w], c)
    tails = CA.alloc_canon_tails(3, taps, D, "cpu").fill_(9.0)
    got, rows = [[], []], []
    for at, n, p in cut_portions(T, cuts, 9):
        b = StepPlan([p]).build(16, [], "cpu")
        xx = x[at:at + n].clone()
        hs = CA.canon_norm(xx, delta[:, at:at + n], coef, tails, b, 1e-3,
                           torch.float32, [False, False])
        rows.append(xx)
        for g, h in zip(got, hs):
            assert h.shape == (n, 32) and not h[:, D:].any()
            g.append(h[:, :D])
    full = (x + delta.sum(0)).double()
    assert torch.allclose(torch.cat(rows).double(), full, atol=1e-5)
    for g, wi, ci in zip(got, w, c):
        ref = oracle.canon(oracle.centered_norm(full, wi.double(), 1e-3),
                           ci.double())
        assert torch.allclose(torch.cat(g).double(), ref, atol=1e-5)
    assert (tails[0] == 9).all() and (tails[2] == 9).all()


@pytest.mark.parametrize("cuts", CUTS)
@pytest.mark.parametrize("window", [None, 1, 7, 16, 40])
@pytest.mark.parametrize("size", [(4, 2, 12, 20, 3), (1, 1, 1, 1, 1),
                                  (6, 3, 8, 5, 6)])
def test_differential_attention(size, window, cuts):
    """Biases, convolutions, both maps, the window and the norm, over the
    paged cache at any cut."""
    H, G, d, e, taps = size
    T, D, r = 70, 24, randn(3)
    lay = QK.QKVLayout(H, G, d, e, maps=2)
    sizes = {"q": H * 2 * d, "k": G * 2 * d, "v": G * e}
    W, x = {}, r(T, D)
    for n, k in sizes.items():
        W[n], W[n + ".b"], W[n + ".conv"] = r(k, D), r(k), r(k, taps)
    for n in ("lq1", "lk1", "lq2", "lk2"):
        W[n] = r(d) * 0.5
    W["o"] = torch.eye(H * e)
    m = {"heads": H, "kv_heads": G, "dim": d, "vdim": e, "conv": taps,
         "diff": 0.3, "scale": 0.4}
    if window is not None:
        m["mask"] = {"size": window}
    W = {k: v.double() for k, v in W.items()}
    ref = oracle.diff_attention(x.double(), W, "", m, 1e-4)
    f = {k: v.float() for k, v in W.items()}
    y = x @ QK.pack_qkv(lay, f["q"], f["k"], f["v"]).T
    bias = QK.pack_qkv(lay, *(f[n + ".b"][:, None] for n in "qkv"))[:, 0]
    conv = QK.pack_qkv(lay, *(f[n + ".conv"] for n in "qkv")).t().contiguous()
    diff = SK.DiffMaps(oracle.lambda_of(W, "", 0.3).float().view(1), e, 1e-4)
    cache = SK.alloc_shared_kv_cache(9, lay, "cpu", torch.float32)
    tails = QK.alloc_conv_tails(3, taps, lay, "cpu", torch.float32)
    tails.fill_(9.0)
    z = torch.zeros(T, lay.n_z)
    for at, n, p in cut_portions(T, cuts, 9):
        b = StepPlan([p]).build(16, [], "cpu")
        q = QK.qkv_conv(y[at:at + n], lay, bias, conv, tails, b, cache)
        run = SK.shared_kv_attend if b.n_short else SK.shared_kv_flash
        run(q, lay, cache, b, 0.4, window, z[at:at + n], out_scale=0.7,
            diff=diff)
    got = z.view(T, H, lay.vc)[..., :e].reshape(T, -1)
    assert torch.allclose(got.double(), ref, atol=2e-4)


@pytest.mark.parametrize("inside", [True, False])
@pytest.mark.parametrize("window", [1, 2, 15, 16, 17, 33])
def test_standout_key_at_the_edge_of_a_window(window, inside):
    """A key that would take the first map's whole output is the last one
    inside the query's window, or the first one outside."""
    H, d, e, query = 2, 4, 6, 50
    lay = QK.QKVLayout(H, 1, d, e, maps=2)
    r = randn(window)
    key = query - window + (1 if inside else 0)
    p = portions((1, query, 0), blocks=9)[0]
    cache = r(9, 1, 16, lay.ec)
    cache[..., lay.voff + e:] = 0                    # padding
    cache[..., d - 1] = cache[..., lay.hc + d - 1] = 0
    cache[p.blocks[key // 16], 0, key % 16, d - 1] = 10.0
    q = torch.zeros(1, 2 * H, lay.hc)
    q[..., d - 1] = 10.0
    z = torch.zeros(1, lay.n_z)
    SK.shared_kv_attend(q.view(1, -1), lay, cache,
                        StepPlan([p]).build(16, [], "cpu"), 1.0, window, z,
                        diff=SK.DiffMaps(torch.tensor([0.5]), e, 1e-6))
    rows = cache[p.blocks, 0, :, lay.voff:lay.voff + e].reshape(-1, e)
    mean = rows[max(0, query - window + 1):query + 1].mean(0)
    first = rows[key] if inside else mean
    ref = oracle.rms((first - 0.5 * mean).double(), 1e-6)
    got = z.view(H, lay.vc)[:, :e].double()
    assert torch.allclose(got, ref.expand(H, e), atol=1e-3)


@pytest.mark.parametrize("cuts", CUTS)
@pytest.mark.parametrize("size", [(3, 12, 20, 28, 36), (1, 1, 1, 1, 1),
                                  (5, 20, 6, 9, 50)])
def test_positionless_latent_attention(size, cuts):
    H, d, e, rq, rank = size
    layer = oracle.latent(H, d, e, rq, rank, scale=0.4)
    cfg = oracle.make_config([layer], 24, 20)
    W = oracle.make_weights(cfg, 1)
    x = randn(5)(70, 24)
    f = {k: v.double() for k, v in W.items()}
    f["l0.mix.o"] = torch.eye(H * e).double()
    ref = oracle.latent_attention(x.double(), f, "l0.mix.", layer["mixer"],
                                  cfg["norm"]["eps"])
    m = load(cfg, W, torch.float32).blocks[0].mixer
    m.fuse()
    y = x @ m.in_rows.T
    cache = m.alloc_cache(9, 3, "cpu")
    z = torch.zeros(70, m.n_o)
    for at, n, p in cut_portions(70, cuts, 9):
        b = StepPlan([p]).build(16, [None], "cpu")
        m(y[at:at + n], b, cache, None, {}, z[at:at + n], None)
    got = z.view(70, H, m.lay.vc)[..., :e].reshape(70, -1)
    assert torch.allclose(got.double(), ref, atol=2e-4)


@pytest.mark.parametrize("cuts", CUTS)
@pytest.mark.parametrize("size", [(3, 20, 6), (1, 1, 1), (2, 16, 40)])
def test_generalized_delta_rule(size, cuts):
    H, d, rank = size
    cfg = oracle.make_config([oracle.delta(H, d)], 24, 20)
    W = oracle.make_weights(cfg, 1, rank=rank)
    x = randn(5)(70, 24)
    f = {k: v.double() for k, v in W.items()}
    f["l0.mix.o"] = torch.eye(H * d).double()
    ref = oracle.general_delta(x.double(), f, "l0.mix.", {"heads": H,
                                                          "dim": d},
                               cfg["norm"]["eps"])
    m = load(cfg, W, torch.float32).blocks[0].mixer
    m.fuse()
    y = x @ m.in_rows.T
    state = m.alloc_cache(9, 3, "cpu").fill_(9.0)
    z = torch.zeros(70, m.n_o)
    for at, n, p in cut_portions(70, cuts, 9):
        b = StepPlan([p]).build(16, [], "cpu")
        m(y[at:at + n], b, state, None, {}, z[at:at + n], None)
    got = z.view(70, H, m.lay.vc)[..., :d].reshape(70, -1)
    assert torch.allclose(got.double(), ref, atol=2e-4)
    assert (state[0] == 9).all() and (state[2] == 9).all()


def test_both_terms_of_the_delta_rule_read_the_old_state():
    """By hand, one channel: S1 = k v; S2 = w S1 - a u (u S1) + k v."""
    lay = GD.GeneralDeltaLayout(1, 1, 1, 1)
    y, y2 = torch.zeros(2, lay.n_y), torch.zeros(2, lay.n_y2)
    y[:, 0] = 1.0                                    # r
    y[:, lay.off_k], y[:, lay.off_v] = 2.0, 3.0
    b = StepPlan(portions((2, 0, 0))).build(16, [], "cpu")
    state, o = GD.alloc_general_delta_state(1, lay, "cpu"), torch.zeros(
        2, lay.n_o)
    GD.general_delta_step(y, y2, lay, torch.zeros(2, 8), -1.0, state, b, o)
    w, a = float(torch.exp(torch.tensor(-0.5))), 0.5
    assert abs(float(o[0, 0]) - 6) < 1e-5
    assert abs(float(o[1, 0]) - (w * 6 - a * 6 + 6)) < 1e-4


@pytest.mark.parametrize("ff", [1, 5, 40])
def test_poly_norm(ff):
    r = randn(ff)
    u, act = r(6, 64) * 2, r(4)
    z = torch.full((6, 64), 7.0)
    PN.poly_norm(u, ff, ff, act, 1e-3, z, 16)
    ref = oracle.poly_norm(u[:, :ff].double(), act.double().tolist(), 1e-3)
    assert torch.allclose(z[:, 16:16 + ff].double(), ref, atol=1e-5)
    assert (z[:, :16] == 7).all() and not z[:, 16 + ff:].any()
    # columns spread over ranks: the sums are the whole token's
    if ff == 40:
        sums = PN.power_sums(u[:, :16], 16) + PN.power_sums(u[:, 16:40], 24)
        part = torch.zeros(6, 32)
        PN.poly_norm(u[:, 16:], 24, 40, act, 1e-3, part, 0, sums=sums)
        assert torch.allclose(part[:, :24].double(), ref[:, 16:], atol=1e-5)


def test_softcap():
    x = randn(0)(2, 3, 9) * 30
    ref = oracle.softcap(x.sum(0).double(), 7.0)
    assert torch.allclose(ops.softcap(x, 7.0).double(), ref, atol=1e-5)


def test_norm_weight_around_zero():
    norm = ops.RMSNorm(12, eps=1e-3, offset=1.0)
    assert not norm.weight.any()
    norm.weight.data.copy_(randn(1)(12))
    x = randn(2)(5, 12)
    ref = oracle.centered_norm(x.double(), norm.weight.double(), 1e-3)
    got = ops.norm_res32(norm, x.clone(), None, torch.float32)
    assert torch.allclose(got.double(), ref, atol=1e-5)
    with pytest.raises(NotImplementedError):
        norm(x)


# --- whole models --------------------------------------------------------------

@pytest.mark.parametrize("name", list(MODELS))
@pytest.mark.parametrize("cuts", [[1000], [1], [2], [3, 40, 2, 1, 17],
                                  [16, 32, 48], [33, 31]])
def test_any_cut_of_the_prompt(name, cuts):
    cfg, W = make(name)
    toks = tokens_of(cfg, 60 if cuts in ([1], [2]) else 150)
    ref = oracle.forward(cfg, W, toks)
    eng = make_engine(cfg, W)
    assert rel_err(run_cut(eng, toks, cuts), ref) < TOL
    assert len(eng.allocator.free) == eng.allocator.num_blocks
    assert sorted(eng.free_slots) == list(range(eng.max_batch))


def test_residual_after_every_layer():
    """Layer by layer, every pass of the loop."""
    cfg, W = make("mixed")
    toks = tokens_of(cfg, 23)
    want = []
    oracle.forward(cfg, W, toks, layers_out=want)
    eng = make_engine(cfg, W)
    got = []
    for blk in eng.model.blocks:
        def step(x, *a, inner=blk.step):
            d = inner(x, *a)
            got.append(x + (d if d.dim() == 2 else d.sum(0)))
            return d
        blk.step = step
    run_cut(eng, toks, [23])
    assert len(got) == len(want) == 9
    for a, b in zip(got, want):
        assert rel_err(a, b) < TOL


def _mixer(c, i):
    return c["layers"][i]["mixer"]


CHANGES = {
    "eps": lambda c: c["norm"].update(eps=0.05),
    "cap": lambda c: c.update(logit_softcap=6.0),
    "no cap": lambda c: c.pop("logit_softcap"),
    "scale": lambda c: _mixer(c, 0).update(scale=0.7),
    "latent scale": lambda c: _mixer(c, 2).update(scale=0.9),
    "difference": lambda c: _mixer(c, 3).update(diff=0.2),
    "window one more": lambda c: _mixer(c, 0)["mask"].update(size=22),
    "window one less": lambda c: _mixer(c, 3)["mask"].update(size=34),
    "no window": lambda c: _mixer(c, 3).pop("mask"),
    "no feed-forward": lambda c: c["layers"][2].update(mlp=None),
    "loop start": lambda c: c["loop"].update(start=2),
    "loop stop": lambda c: c["loop"].update(stop=5),
    "one pass": lambda c: c["loop"].update(times=1),
    "no loop": lambda c: c.pop("loop"),
}


@pytest.mark.parametrize("change", list(CHANGES))
def test_every_constant_is_read(change):
    """Each constant, and each window by one token, shows in the oracle far
    beyond the tolerance that the engine keeps."""
    cfg, W = make("mixed")
    toks = tokens_of(cfg, 90)
    ref = oracle.forward(cfg, W, toks)
    CHANGES[change](cfg)
    if change == "one pass":
        W["loop.step"] = W["loop.step"][:1]
    drop = {"no feed-forward": ("l2.mlp", "l2.norm2", "l2.canon2"),
            "no loop": ("loop.",)}.get(change)
    W = {k: v for k, v in W.items() if not drop or not k.startswith(drop)}
    moved = oracle.forward(cfg, W, toks)
    assert rel_err(moved, ref) > 30 * TOL
    assert rel_err(run_cut(make_engine(cfg, W), toks, [25]), moved) < 3 * TOL


def test_every_tensor_counts():
    cfg, W = make("mixed")
    toks = tokens_of(cfg, 40)
    ref = oracle.forward(cfg, W, toks)
    for name in W:
        if name == "embed" or W[name].dim() == 2 and min(W[name].shape) > 6:
            continue                       # plain products show elsewhere
        V = dict(W)
        V[name] = (W[name].float() * 0.5 - 0.2).flip(0).to(W[name].dtype)
        moved = oracle.forward(cfg, V, toks)
        assert rel_err(moved, ref) > 50 * TOL, name
        assert rel_err(run_cut(make_engine(cfg, V), toks, [25]),
                       moved) < 3 * TOL, name


def test_first_tokens_and_single_token_prompt():
    for name in ("mixed", "recurrent"):
        cfg, W = make(name)
        for n in (1, 2, 3, 5, 7):
            toks = tokens_of(cfg, n, seed=n)
            ref = oracle.forward(cfg, W, toks)
            for cuts in ([n], [1], [2, 1]):
                assert rel_err(run_cut(make_engine(cfg, W), toks, cuts),
                               ref) < TOL


@pytest.mark.parametrize("name", ["recurrent", "mixed"])
def test_a_token_far_back(name):
    """One early token changes logits far behind it, through a state or the
    latent attention, and the engine follows."""
    cfg, W = make(name)
    for k in W:
        if k.endswith(".w0"):              # states that forget slowly
            W[k] = W[k] - 6
        elif k.endswith(".a.b"):
            W[k] = W[k] - 4
    a = tokens_of(cfg, 300)
    b = [(a[0] + 1) % cfg["vocab"]] + a[1:]
    ra, rb = (oracle.forward(cfg, W, t)[-20:] for t in (a, b))
    assert rel_err(ra, rb) > 30 * TOL
    for toks, ref in ((a, ra), (b, rb)):
        got = run_cut(make_engine(cfg, W), toks, [200, 64, 1])
        assert rel_err(got[-20:], ref) < TOL


def test_a_query_finds_one_key_among_hundreds():
    """One head's query and one key share a direction that no other has, so
    that the score stands out at any distance."""
    layers = [oracle.latent(2, 8, 8, 24, 24, scale=1.0)]
    cfg = oracle.make_config(layers, 24, 40, taps=2, cap=None)
    W = oracle.make_weights(cfg, 2)
    # a part of the query that every token has, and of the key that one has
    W["embed"][:, :2] = torch.tensor([2.0, 0.0])
    W["embed"][39, 1] = 8.0
    for n, col in (("q", 0), ("kv", 1)):
        W[f"l0.mix.d{n}"][0] = 3.0 * (torch.arange(24) == col)
        W[f"l0.mix.u{n[0]}"][0] = 4.0 * (torch.arange(24) == 0)
    toks = [t % 39 for t in tokens_of(cfg, 400)]
    for at in (0, 1, 15, 16, 200, 397):
        marked = list(toks)
        marked[at] = 39
        ref = oracle.forward(cfg, W, marked)
        plain = oracle.forward(cfg, W, toks)
        assert rel_err(ref[-1:], plain[-1:]) > 30 * TOL
        got = run_cut(make_engine(cfg, W), marked, [300, 90, 1])
        assert rel_err(got, ref) < 2 * TOL


@pytest.mark.parametrize("name", ["mixed", "windows", "recurrent"])
def test_unequal_requests_in_one_batch(name):
    """Portions beside single tokens, requests that pause, end and make way:
    every logit as if the request were alone, on a pool that only just holds
    the live ones."""
    cfg, W = make(name)
    lens = [90, 3, 61, 1, 97, 40]
    seqs = [tokens_of(cfg, n, seed=i) for i, n in enumerate(lens)]
    refs = [oracle.forward(cfg, W, s) for s in seqs]
    eng = make_engine(cfg, W, kv_blocks=23, max_batch=3)
    g = torch.Generator().manual_seed(5)
    waiting, live, owners = list(range(len(seqs))), {}, {}
    while waiting or live:
        while waiting and len(live) < 3:
            i = waiting.pop(0)
            live[i] = [eng.open_request(), 0]
        entries, ids = [], []
        for i, (r, at) in live.items():
            if len(live) > 1 and int(torch.randint(0, 4, (1,),
                                                   generator=g)) == 0:
                continue
            n = [1, 1, 2, 7, 34, 50][int(torch.randint(0, 6, (1,),
                                                       generator=g))]
            n = min(n, len(seqs[i]) - at)
            entries.append((r, seqs[i][at:at + n], range(n)))
            ids.append((i, at, n))
        if not entries:
            continue
        logits = eng.run_portions(entries)
        row = 0
        for (i, at, n), (r, _, _) in zip(ids, entries):
            assert rel_err(logits[row:row + n], refs[i][at:at + n]) < 3 * TOL
            row += n
            live[i][1] = at + n
            owners.setdefault(r.slot, set()).add(i)
            if at + n == len(seqs[i]):
                eng.close_request(r)
                del live[i]
    assert len(owners) == 3 and max(len(o) for o in owners.values()) > 1
    assert len(eng.allocator.free) == eng.allocator.num_blocks
    assert sorted(eng.free_slots) == [0, 1, 2]


def _tensors(cache):
    if torch.is_tensor(cache):
        return [cache]
    return [t for c in cache for t in _tensors(c)]


def test_stale_pages_and_slots_do_not_leak():
    cfg, W = make("mixed")
    eng = make_engine(cfg, W, kv_blocks=12)
    toks = tokens_of(cfg, 100, seed=8)
    ref = oracle.forward(cfg, W, toks)
    for t in _tensors(eng.caches):
        t.fill_(50.0)
    assert rel_err(run_cut(eng, toks, [7, 1, 40]), ref) < TOL
    assert rel_err(run_cut(eng, toks, [50]), ref) < TOL
    assert rel_err(run_cut(eng, toks, [1, 2]), ref) < TOL


def test_every_layer_run_has_a_cache_of_its_own():
    cfg, W = make("mixed")
    eng = make_engine(cfg, W)
    assert eng.model.runs == [(0, None), (1, 0), (2, None), (3, None), (1, 1),
                              (2, None), (3, None), (4, None), (5, None)]
    tensors = _tensors(eng.caches)
    assert len({t.data_ptr() for t in tensors}) == len(tensors) == 21
    (kv, conv), canon = eng.caches[0]
    assert kv.shape == (128, 2, 16, 2 * 24 + 32)
    assert conv.shape == (7, 1, (12 + 4) * 24 + 2 * 32)
    assert canon.shape == (7, 3, 48) and canon.dtype == torch.float32
    S, _ = eng.caches[1]
    assert S.shape == (7, 3, 24, 24) and S.dtype == torch.float32
    assert eng.caches[2][0].shape == (128, 16, 40)     # latents only
    per_slot = sum(t[0].numel() * t.element_size() for t in tensors
                   if t.shape[0] == 7)
    assert eng.model.state_bytes() == per_slot
    per_block = sum(t[0].numel() * t.element_size() for t in tensors
                    if t.shape[0] == 128)
    assert eng.model.kv_bytes_per_block() == per_block


def test_cache_is_bounded_by_the_widest_window():
    cfg, W = make("windows")
    eng = make_engine(cfg, W)
    r = eng.open_request()
    run_cut(eng, tokens_of(cfg, 300), [50, 1, 1], req=r)
    assert r.dropped > 220 and len(r.blocks) * 16 <= 26 + 50 + 32
    cfg, W = make("mixed")                 # latent attention sees everything
    full = make_engine(cfg, W)
    r = full.open_request()
    run_cut(full, tokens_of(cfg, 150), [64], req=r)
    assert r.dropped == 0
    cfg, W = make("recurrent")             # nothing is cached at all
    rec = make_engine(cfg, W)
    r = rec.open_request()
    run_cut(rec, tokens_of(cfg, 100), [9], req=r)
    assert len(r.blocks) <= 2


# --- scheduler ------------------------------------------------------------------

def _assert_greedy(cfg, W, req, prompt, n):
    ids = req.prompt_ids + req.output_ids
    assert ids[:len(prompt)] == prompt and len(ids) == len(prompt) + n
    ref = oracle.forward(cfg, W, ids).argmax(-1).tolist()
    assert ref[len(prompt) - 1:-1] == ids[len(prompt):]


def test_greedy_generation_long():
    cfg, W = make("mixed")
    eng = make_engine(cfg, W)
    prompt = tokens_of(cfg, 30)
    out = eng.generate(prompt, max_new_tokens=120)
    ref = oracle.forward(cfg, W, prompt + out).argmax(-1).tolist()
    assert ref[29:-1] == out


@pytest.mark.parametrize("chunk,blocks", [(2048, 128), (20, 24), (200, 13)])
def test_scheduler_batches(chunk, blocks):
    """Admission, prompt portions beside decoding, preemption on a small
    pool: the greedy continuation never changes."""
    cfg, W = make("mixed")
    eng = make_engine(cfg, W, kv_blocks=blocks, max_batch=3)
    assert not eng.prefix_cache_enabled    # blocks alone are not the state
    eng.prefill_chunk = chunk
    base = tokens_of(cfg, 100, seed=4)
    prompts = [base[:n] for n in (1, 60, 100, 33)] + \
        [tokens_of(cfg, 70, seed=9)]
    reqs = [eng.submit(p, max_new_tokens=20) for p in prompts]
    steps = 0
    while eng.has_work():
        eng.step()
        steps += 1
        assert steps < 2000
    for r, p in zip(reqs, prompts):
        _assert_greedy(cfg, W, r, p, 20)
    if blocks == 13:
        assert eng.stats["preemptions"] > 0
    assert len(eng.allocator.free) == eng.allocator.num_blocks
    assert sorted(eng.free_slots) == [0, 1, 2]


# --- configuration, weights, command line -------------------------------------

def test_checkpoint_directory_round_trip(tmp_path):
    cfg, W = make("mixed")
    d = write_checkpoint(tmp_path / "m", cfg, W)
    mc = config_from_dir(d)
    back = config_from_dopilorn(config_to_dopilorn(mc), shapes_of(W))
    assert back.layers == mc.layers and back.loop == mc.loop
    assert mc.loop == LoopSpec(1, 4, 2, step=True)
    assert (back.canon, back.logit_softcap, back.norm_offset) == (4, 20.0, 1.0)
    assert mc.layers[1].mixer.decay_rank == 6      # from the tensors
    assert mc.sliding_window is None and mc.norm_eps == 2e-5
    assert mc.kernel_groups == ("core", "delta", "dual", "latent",
                                "shared_kv")
    m = build_model(mc, dtype=torch.float32)
    load_pretrained(m, d)
    ref = load(cfg, W, torch.float32)
    for (k, a), (_, b) in zip(m.state_dict().items(),
                              ref.state_dict().items()):
        assert torch.equal(a, b), k
    del W["l2.canon1"]
    with pytest.raises(KeyError):
        load_pretrained(build_model(mc, dtype=torch.float32),
                        write_checkpoint(tmp_path / "bad", cfg, W))


def test_configuration_errors():
    cfg, W = make("mixed")
    shapes = shapes_of(W)

    def broken(f):
        c = json.loads(json.dumps(cfg))
        f(c)
        return c
    for f in (lambda c: c["layers"][0].update(type="other"),
              lambda c: c["layers"][0]["mlp"].update(kind="moe"),
              lambda c: _mixer(c, 0).update(kv_heads=4),
              lambda c: _mixer(c, 0).update(conv=0),
              lambda c: _mixer(c, 0)["mask"].update(size=0),
              lambda c: _mixer(c, 2).update(q_rank=0),
              lambda c: c["canon"].update(taps=0),
              lambda c: c.update(logit_softcap=0.0),
              lambda c: c["loop"].update(stop=9)):
        with pytest.raises(ValueError):
            config_from_dopilorn(broken(f), shapes)
    with pytest.raises(ValueError, match="no tensor"):
        config_from_dopilorn(cfg, {})
    for where in (lambda c: c, lambda c: _mixer(c, 0),
                  lambda c: _mixer(c, 1), lambda c: _mixer(c, 2),
                  lambda c: c["canon"], lambda c: c["loop"]):
        c = broken(lambda c: where(c).update(extra=1))
        with pytest.warns(UserWarning, match="without effect"):
            config_from_dopilorn(c, shapes)


def test_registry_and_packing_keep_parameters():
    mc = get_config("tiny-dopilorn")
    m = build_model(mc, dtype=torch.float32)
    before = {k: v.clone() for k, v in m.state_dict().items()}
    for blk in m.blocks:
        blk.fuse()
    for k, v in m.state_dict().items():
        assert torch.equal(v, before[k]), k
    assert mc.params_b > 0 and len(m.blocks) == 4
    # one differential attention, one latent layer that runs twice
    assert m.kv_bytes_per_block() == (2 * (2 * 16 + 24) + 2 * 24) * 16 * 4


def test_parts_serve_another_design():
    """Plain norms, no loop, no cap, a slower decay, one kind of mixer or
    several: the same blocks under another description."""
    layers = [LayerSpec(GeneralDeltaSpec(2, 4, 3, decay_scale=-0.1), None),
              LayerSpec(LatentAttentionSpec(2, 4, 0, 6, 8, 0.5, q_rank=8,
                                            head_gate=True), PolyNormSpec(7)),
              LayerSpec(DiffAttentionSpec(2, 1, 4, 4, 0.5, 0.0, 1),
                        PolyNormSpec(12))]
    toks = [3, 1, 4, 1, 5, 9, 2, 6]
    for some in (layers, layers[1:], layers[2:]):
        mc = layered_config("p", some, 16, 20, max_seq_len=64, canon=1)
        assert mc.layout == "dual"
        eng = Engine(mc, dtype=torch.float32, device="cpu", kv_blocks=16)
        whole = run_cut(eng, toks, [8])
        assert torch.allclose(whole, run_cut(eng, toks, [1]), atol=1e-5)
    for bad in (dict(), dict(canon=2, streams=2, norm="dyt"),
                dict(canon=2, norm="layernorm")):
        with pytest.raises(ValueError):
            layered_config("q", layers, 16, 20, **bad)
    with pytest.raises(ValueError, match="mlp"):
        layered_config("r", [LayerSpec(layers[0].mixer, GLUSpec(8))], 16, 20,
                       canon=2)
    with pytest.raises(ValueError, match="layout"):
        layered_config("s", [LayerSpec(get_config("tiny-keralorn").layers[0]
                                       .mixer, None)], 16, 20, canon=2)


def test_synthetic_model_loads_and_serves(tmp_path):
    from runbooks_amd.workloads.model_loader import materialize_synthetic
    materialize_synthetic("tiny-dopilorn", tmp_path)
    mc = config_from_dir(tmp_path)
    m = load_pretrained(build_model(mc, dtype=torch.float32, seed=5),
                        tmp_path)
    out = Engine(m, device="cpu", kv_blocks=32).generate([1, 2, 3], 5)
    assert len(out) == 5


def test_http_server_serves_the_family():
    from fastapi.testclient import TestClient
    from runbooks_amd.serve import ByteTokenizer
    from runbooks_amd.serve.http import build_app
    eng = Engine("tiny-dopilorn", device="cpu", dtype=torch.float32,
                 kv_blocks=64)
    with TestClient(build_app(eng, ByteTokenizer(),
                              model_name="tiny-dopilorn")) as client:
        r = client.post("/v1/completions", json={
            "prompt": "hello", "max_tokens": 4, "temperature": 0.0})
        assert r.status_code == 200
        assert r.json()["usage"]["completion_tokens"] == 4


def test_fp8_cache_and_training_are_refused():
    with pytest.raises(NotImplementedError, match="fp8"):
        make_engine(*make("mixed"), kv_fp8=True)
    with pytest.raises(NotImplementedError, match="serving only"):
        load(*make("mixed"), torch.float32)(torch.zeros(1, 3).long())


def test_replay_command(tmp_path, capsys, monkeypatch):
    from runbooks_amd.serve.replay import main
    cfg, W = make("mixed")
    d = write_checkpoint(tmp_path / "m", cfg, W)
    a, b = tokens_of(cfg, 60, 1), tokens_of(cfg, 9, 2)
    steps = [
        {"step": 0, "entries": [{"id": "a", "tokens": a[:40],
                                 "want": [0, 39]}], "end": []},
        {"step": 1, "entries": [{"id": "b", "tokens": b[:8], "want": []}],
         "end": []},
        {"step": 2, "entries": [{"id": "b", "tokens": b[8:], "want": [0]},
                                {"id": "a", "tokens": a[40:], "want": [19]}],
         "end": ["a", "b"]},
        {"step": 3, "entries": [{"id": "a", "tokens": b, "want": [8]}],
         "end": ["a"]}]
    monkeypatch.setattr("sys.stdin", io.StringIO(
        "".join(json.dumps(s) + "\n" for s in steps)))
    out = tmp_path / "out"
    out.mkdir()
    assert main(["--model", str(d), "--dtype", "float32", "--out", str(out),
                 "--max-tokens", "128", "--device", "cpu"]) == 0
    assert [ln for ln in capsys.readouterr().out.splitlines()
            if ln.startswith("done")] == [f"done {i}" for i in range(4)]
    ra, rb = oracle.forward(cfg, W, a), oracle.forward(cfg, W, b)
    want = {0: ra[[0, 39]], 2: torch.stack([rb[8], ra[59]]), 3: rb[8:]}
    assert sorted(os.listdir(out)) == ["0.f32", "2.f32", "3.f32"]
    for k, ref in want.items():
        got = torch.from_numpy(np.fromfile(out / f"{k}.f32", dtype="<f4"))
        assert rel_err(got.view(ref.shape), ref) < TOL
