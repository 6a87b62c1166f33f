"""The Keralorn family on the CPU path: every op and whole engine runs
against the plain oracle (tests/keralorn_oracle.py)."""
import io
import json
import os

import numpy as np
import pytest
import torch

import keralorn_oracle as oracle
from keralorn_helpers import (MODELS, load, make, make_engine, portions,
                              rel_err, run_cut, tokens_of, write_checkpoint)
from runbooks_amd import ops
from runbooks_amd.models import build_model, get_config
from runbooks_amd.models.config import (GLUSpec, LayerSpec, LightningSpec,
                                        LoopSpec, RopeScaling,
                                        SharedKVAttentionSpec, layered_config)
from runbooks_amd.models.load import (config_from_dir, config_from_keralorn,
                                      config_to_keralorn, load_pretrained)
from runbooks_amd.models.ragged import StepPlan
from runbooks_amd.ops import lightning as LA
from runbooks_amd.ops import shared_kv as SK
from runbooks_amd.serve import Engine

TOL = 2e-5


# --- single mechanisms -------------------------------------------------------

def test_layer_norm_and_join_on_a_32_bit_residual():
    g = torch.Generator().manual_seed(0)
    x = torch.randn(5, 24, generator=g) + 7
    d, other = torch.randn(2, 5, 24, generator=g)
    w, b = torch.rand(2, 24, generator=g)
    for delta, add in ((None, 0), (d, d), (torch.stack([d, d]), 2 * d)):
        y = x.clone()
        joined = ops.join_res32(y, delta, other)
        assert torch.equal(y, x)
        assert torch.allclose(joined, torch.cat([x + add, other], -1))
        got = ops.layernorm_res32(y, delta, w, b, 3e-3, torch.float32)
        assert torch.allclose(y, x + add)
        ref = oracle.layer_norm((x + add).double(), w.double(), b.double(),
                                3e-3)
        assert torch.allclose(got.double(), ref, atol=1e-5)


@pytest.mark.parametrize("dims", [2, 6, 16])
@pytest.mark.parametrize("scaling", [
    None, (8.0, 1.0, 4.0, 64.0), (3.0, 0.5, 2.0, 1000.0),
    (2.0, 1.0, 1.0, 20.0), (4.0, 1.0, 4.0, 1e9), (4.0, 1.0, 4.0, 1e-3)])
def test_rotation_in_halves_with_scaled_frequencies(dims, scaling):
    rot = {"base": 777.0, "dims": dims}
    spec = None
    if scaling:
        rot["scaling"] = dict(zip(("factor", "low", "high", "original"),
                                  scaling))
        spec = RopeScaling(*scaling)
    f = ops.rope_frequencies(dims, 777.0, spec)
    assert torch.allclose(f, torch.tensor(oracle.rotation_frequencies(rot),
                                          dtype=torch.float64), rtol=1e-12)
    x = torch.randn(7, 3, 18)
    pos = torch.tensor([0, 1, 5, 900, 17, 2, 63])
    cos, sin = ops.rope_tables(dims, 1000, 777.0, freq_scaling=spec)
    got = SK.rotate_halves_ref(x, cos, sin, pos)
    ref = oracle.rotate_halves(x.double(), pos, rot)
    assert torch.allclose(got.double(), ref, atol=1e-5)
    assert torch.equal(got[0], x[0])             # position 0 does not turn
    assert torch.equal(got[..., dims:], x[..., dims:])


def test_scaled_frequencies_cover_all_three_ranges():
    s = RopeScaling(8.0, 1.0, 4.0, 64.0)
    plain = ops.rope_frequencies(16, 10000.0)
    f = ops.rope_frequencies(16, 10000.0, s)
    wave = 2 * np.pi / plain
    keep, stretch = wave < 16, wave > 64
    assert keep.any() and stretch.any() and (~keep & ~stretch).any()
    assert torch.equal(f[keep], plain[keep])
    assert torch.allclose(f[stretch], plain[stretch] / 8)
    mid = ~keep & ~stretch
    assert ((f[mid] < plain[mid]) & (f[mid] > plain[mid] / 8)).all()


def test_gated_gelu():
    g = torch.tensor([[-9.0, -0.5, 0.0, 1.1, 8.0]])
    u = torch.tensor([[5.0, -7.0, 0.2, -0.4, 0.9]])
    got = ops.geglu(torch.cat([g, u], 1))
    assert torch.allclose(got.double(),
                          oracle.gelu_tanh(g.double()) * u.double(),
                          atol=1e-6)


@pytest.mark.parametrize("H,G,dim,rot", [(6, 2, 20, 12), (2, 2, 16, 16),
                                         (3, 1, 7, 2), (4, 1, 8, 0)])
def test_projection_layout_and_cached_rows(H, G, dim, rot):
    """The padded joint product and its epilogue give the oracle's queries;
    a cached row is key and value at once; the output weight undoes the
    value's order."""
    lay, D, T = SK.SharedKVLayout(H, G, dim, rot), 40, 9
    g = torch.Generator().manual_seed(1)
    q, k = (torch.randn(n * dim, D, generator=g) for n in (H, G))
    h = torch.randn(T, D, generator=g) * 0.2
    pos = torch.arange(T, dtype=torch.int32) + 4
    slots = torch.tensor([40, 3, 17, 16, 15, 31, 32, 5, 63],
                         dtype=torch.int32)
    cos, sin = ops.rope_tables(rot, 64, 100.0)
    y = h @ SK.pack_in(lay, q, k).T
    cache = SK.alloc_shared_kv_cache(4, lay, "cpu", torch.float32)
    SK.shared_kv_prep(y, lay, cos, sin, pos, slots, cache)
    r = {"base": 100.0, "dims": rot}

    def unpad(x):                        # [.., hc] -> [.., dim]
        return torch.cat([x[..., :rot],
                          x[..., lay.rotc:lay.rotc + dim - rot]], -1)
    qq = (h.double() @ q.double().T).view(T, H, dim)
    kk = (h.double() @ k.double().T).view(T, G, dim)
    got = unpad(y[:, :lay.off_k].view(T, H, lay.hc)).double()
    assert torch.allclose(got, oracle.rotate_halves(qq, pos, r), atol=1e-5)
    s = slots.long()
    rows = cache[s // 16, :, s % 16].double()
    assert torch.allclose(unpad(rows), oracle.rotate_halves(kk, pos, r),
                          atol=1e-5)
    value = rows[..., lay.rotc:]
    o = torch.randn(D, G * dim, generator=g)
    vl = SK.SharedKVLayout(G, G, dim, rot)
    z = torch.zeros(T, vl.n_z, dtype=torch.float64)
    z[:, :G * lay.hc] = value.reshape(T, -1)
    assert torch.allclose(z @ SK.pack_out(vl, o).double().T,
                          kk.reshape(T, -1) @ o.double().T, atol=1e-4)
    untouched = torch.ones(4, 16, dtype=torch.bool)
    untouched[s // 16, s % 16] = False
    assert not cache.transpose(1, 2)[untouched].any()


def _attention_case(window, ps, peak=None, seed=0):
    """One batch through the op, and the oracle's answer. peak (sequence,
    query, key): that query scores the key far above all others."""
    H, G, dim, rot = 4, 2, 12, 8
    lay = SK.SharedKVLayout(H, G, dim, rot)
    g = torch.Generator().manual_seed(seed)
    T = sum(len(p.tokens) for p in ps)
    cache = torch.zeros(64, G, 16, lay.ec)
    cache[..., :dim] = torch.randn(64, G, 16, dim, generator=g)
    cache[..., lay.hc:] = torch.randn(64, G, 16, lay.rotc, generator=g)
    q = torch.randn(T, H, lay.hc, generator=g)
    q[..., dim:] = 0
    first = [sum(len(p.tokens) for p in ps[:i]) for i in range(len(ps))]
    if peak is not None:
        s, query, key = peak
        cache[ps[s].blocks[key // 16], :, key % 16, dim - 1] = 12.0
        q[first[s] + query - (ps[s].start - ps[s].dropped), :, dim - 1] = 12.0
    y = torch.zeros(T, lay.n_y)
    y[:, :lay.off_k] = q.view(T, -1)
    ref = []
    for p, r0 in zip(ps, first):
        n = p.start - p.dropped + len(p.tokens)
        i = torch.arange(n)
        rows = cache[torch.tensor(p.blocks)[i // 16], :, i % 16].double()
        of = [h // 2 for h in range(H)]
        qq = torch.zeros(n, H, lay.hc, dtype=torch.float64)
        qq[n - len(p.tokens):] = q[r0:r0 + len(p.tokens)].double()
        o = oracle.softmax_attention(
            qq, rows[:, of, :lay.hc], rows[:, of, lay.rotc:], 0.21,
            oracle.window_mask(n, window))
        ref.append(o[n - len(p.tokens):].reshape(len(p.tokens), -1))
    b = StepPlan(ps).build(16, [], "cpu")
    z = torch.zeros(T, lay.n_z)
    # the batch's own order: short portions first
    order = torch.cat([torch.arange(r0, r0 + len(p.tokens))
                       for short in (True, False)
                       for p, r0 in zip(ps, first)
                       if (len(p.tokens) <= 32) == short])
    SK.shared_kv_attend(y[order], lay, cache, b, 0.21, window, z)
    SK.shared_kv_flash(y[order], lay, cache, b, 0.21, window, z)
    out = torch.zeros_like(z)
    out[order] = z
    return out, torch.cat(ref), first


@pytest.mark.parametrize("window", [None, 1, 7, 16, 33])
def test_attention_of_any_portion(window):
    drop = 0 if window is None else 16
    ps = portions((1, 0, 0), (5, 0, 0), (1, 47, 0), (40, 60, drop),
                  (2, 15, 0), (17, 16, 0), blocks=64)
    out, ref, _ = _attention_case(window, ps)
    assert (out.double() - ref).abs().max() < TOL


@pytest.mark.parametrize("window,inside", [(20, True), (20, False),
                                           (None, True)])
@pytest.mark.parametrize("query", [31, 32, 47, 70])
def test_standout_key_at_the_window_edge(window, inside, query):
    """A key whose score stands out, just inside or just outside the window
    (or at the very start without one)."""
    ps = portions((40, 40, 0), (60, 20, 0), blocks=64)
    key = 0 if window is None else query - window + (1 if inside else 0)
    out, ref, first = _attention_case(window, ps, peak=(1, query, key))
    assert (out.double() - ref).abs().max() < TOL
    plain, _, _ = _attention_case(window, ps)
    t = first[1] + query - 20
    moved = (out[t] - plain[t]).abs().max()
    assert moved > 1e-1 if inside else True


@pytest.mark.parametrize("decay", [(0.3, 0.9, 0.999), (0.0, 1.0, 0.5)])
def test_recurrence_forms(decay):
    """Token after token, in chunks, and any mixture with the state carried
    between: the oracle's results; a first portion ignores its slot."""
    H, d, e, N = 3, 10, 6, 200
    lay = LA.LightningLayout(H, d, e)
    g = torch.Generator().manual_seed(0)
    q, k, v = (torch.randn(N, H, n, generator=g) for n in (d, d, e))
    y = torch.zeros(N, lay.n_y)
    y[:, :lay.off_k].view(N, H, lay.dc)[..., :d] = q
    y[:, lay.off_k:lay.off_v].view(N, H, lay.dc)[..., :d] = k
    y[:, lay.off_v:lay.off_g].view(N, H, lay.vc)[..., :e] = v
    ref = oracle.linear_recurrence(*(oracle.silu(x.double())
                                     for x in (q, k, v)), decay)
    powers = LA.decay_powers(decay)
    for cuts in ([200], [1], [64, 33, 2], [65, 1, 63, 40]):
        state = torch.full((4, H, lay.dc, lay.vc), 5.0)
        at, i, out = 0, 0, []
        while at < N:
            n = min(cuts[i % len(cuts)], N - at)
            p = portions((n, at, 0))
            p[0].slot = 2
            b = StepPlan(p).build(16, [], "cpu")
            o = torch.zeros(n, lay.n_o)
            LA.lightning_step(y[at:at + n], lay, state, b, powers, o)
            LA.lightning_chunk(y[at:at + n], lay, state, b, powers, o)
            out.append(o.view(n, H, lay.vc)[..., :e])
            at, i = at + n, i + 1
        err = (torch.cat(out).double() - ref).abs().max() / ref.abs().max()
        assert err < TOL
        assert (state[[0, 1, 3]] == 5).all()


def test_norm_over_all_heads_with_gate():
    H, e, T = 3, 6, 5
    lay = LA.LightningLayout(H, 4, e)
    g = torch.Generator().manual_seed(0)
    o = torch.randn(T, H, e, generator=g)
    gate = torch.randn(T, H, e, generator=g)
    w = torch.rand(H * e, generator=g)
    y = torch.zeros(T, lay.n_y)
    y[:, lay.off_g:lay.off_g + lay.n_o].view(T, H, lay.vc)[..., :e] = gate
    op = torch.nn.functional.pad(o, (0, lay.vc - e)).view(T, -1)
    z = torch.full((T, lay.n_z), 3.0)
    LA.lightning_out(op, lay, LA.pack_norm(lay, w), y, z, H * e, 1e-2)
    ref = oracle.rms_norm(o.reshape(T, -1).double(), w.double(), 1e-2) * \
        torch.sigmoid(gate.reshape(T, -1).double())
    w_o = torch.randn(7, H * e, generator=g)
    got = z.double() @ LA.pack_out(lay, w_o).double().T
    assert torch.allclose(got, ref @ w_o.double().T, atol=1e-5)


# --- whole models -------------------------------------------------------------

@pytest.mark.parametrize("name", list(MODELS))
@pytest.mark.parametrize("cuts", [[1000], [1], [2], [3, 40, 2, 1, 17],
                                  [33, 1], [64, 5]])
def test_any_cut_of_the_prompt(name, cuts):
    cfg, W = make(name)
    toks = tokens_of(cfg, 70 if name in ("wide", "big") else 130)
    ref = oracle.forward(cfg, W, toks)
    eng = make_engine(cfg, W)
    assert rel_err(run_cut(eng, toks, cuts), ref) < TOL
    assert len(eng.allocator.free) == eng.allocator.num_blocks
    assert sorted(eng.free_slots) == list(range(eng.max_batch))


def test_bf16_runs_both_forms_of_every_mixer():
    """bf16 on the CPU takes the long-portion forms, too."""
    cfg, W = make("full")
    toks = tokens_of(cfg, 150)
    ref = oracle.forward(cfg, W, toks)
    eng = make_engine(cfg, W, torch.bfloat16)
    assert all(b.expandable for b in eng.model.blocks)
    whole = run_cut(eng, toks, [1000])
    cut = run_cut(eng, toks, [1, 40, 20, 33])
    assert rel_err(whole, ref) < 0.1 and rel_err(cut, ref) < 0.1


def test_residual_after_every_layer_run():
    cfg, W = make("mixed")
    toks = tokens_of(cfg, 70)
    want = []
    oracle.forward(cfg, W, toks, layers_out=want)
    eng = make_engine(cfg, W)
    got = []
    for blk in eng.model.blocks:
        def spy(x, delta, *a, _step=blk.step):
            out = _step(x, delta, *a)
            got.append(x + out)
            return out
        blk.step = spy
    run_cut(eng, toks, [1000])
    assert len(got) == len(want) == 5 + 3
    for g, w in zip(got, want):
        assert (g.double() - w).abs().max() < 1e-4


CHANGES = {
    "window 0 up": lambda c: c["layers"][0]["mixer"]["mask"].update(size=22),
    "window 0 down": lambda c: c["layers"][0]["mixer"]["mask"].update(size=20),
    "window 2 up": lambda c: c["layers"][2]["mixer"]["mask"].update(size=36),
    "window 4 down": lambda c: c["layers"][4]["mixer"]["mask"].update(size=63),
    "scale": lambda c: c["layers"][2]["mixer"].update(scale=0.41),
    "eps": lambda c: c["norm"].update(eps=2e-3),
    "base": lambda c: c["layers"][0]["mixer"]["rot"].update(base=510.0),
    "rotated dims": lambda c: c["layers"][4]["mixer"]["rot"].update(dims=6),
    "factor": lambda c: c["layers"][0]["mixer"]["rot"]["scaling"].update(
        factor=9.0),
    "low": lambda c: c["layers"][0]["mixer"]["rot"]["scaling"].update(
        low=1.2),
    "high": lambda c: c["layers"][0]["mixer"]["rot"]["scaling"].update(
        high=4.4),
    "original": lambda c: c["layers"][0]["mixer"]["rot"]["scaling"].update(
        original=70),
    "no scaling": lambda c: c["layers"][0]["mixer"]["rot"].pop("scaling"),
    "decay": lambda c: c["layers"][1]["mixer"].update(
        decay=[0.35, 0.91, 0.995]),
    "order of decays": lambda c: c["layers"][1]["mixer"].update(
        decay=[0.9, 0.35, 0.995]),
    "one more pass": lambda c: c["loop"].update(times=3),
    "loop start": lambda c: c["loop"].update(start=2),
    "loop stop": lambda c: c["loop"].update(stop=3),
    "no mlp": lambda c: c["layers"][3].update(mlp=None),
}


@pytest.mark.parametrize("change", list(CHANGES))
def test_every_constant_is_read(change):
    """Each constant, and each window by one token, shows in the oracle far
    beyond the tolerance that the engine keeps."""
    cfg, W = make("mixed")
    toks = tokens_of(cfg, 130)
    ref = oracle.forward(cfg, W, toks)
    CHANGES[change](cfg)
    moved = oracle.forward(cfg, W, toks)
    assert rel_err(moved, ref) > 30 * TOL
    if change == "no mlp":
        W = {k: v for k, v in W.items()
             if not k.startswith(("l3.mlp", "l3.norm2"))}
    assert rel_err(run_cut(make_engine(cfg, W), toks, [25]), moved) < 3 * TOL


@pytest.mark.parametrize("drop", ["l0.norm1.b", "final.norm.b", "l1.mix.norm"])
def test_biases_and_weights_of_norms_count(drop):
    cfg, W = make("mixed")
    toks = tokens_of(cfg, 40)
    ref = oracle.forward(cfg, W, toks)
    W[drop] = torch.zeros_like(W[drop]) + (0 if drop.endswith(".b") else 1)
    moved = oracle.forward(cfg, W, toks)
    assert rel_err(moved, ref) > 100 * TOL
    assert rel_err(run_cut(make_engine(cfg, W), toks, [25]), moved) < 3 * TOL


def test_first_tokens_and_single_token_prompt():
    cfg, W = make("mixed")
    for n in (1, 2, 3):
        toks = tokens_of(cfg, n, seed=n)
        ref = oracle.forward(cfg, W, toks)
        for cuts in ([n], [1]):
            assert rel_err(run_cut(make_engine(cfg, W), toks, cuts), ref) < TOL


@pytest.mark.parametrize("name", ["recurrent", "full"])
def test_a_token_far_back(name):
    """One early token changes logits far behind it, through the state (or
    the layer without a window), and the engine follows."""
    cfg, W = make(name)
    for lay in cfg["layers"]:
        if lay["type"] == "lightning":
            lay["mixer"]["decay"][-1] = 0.9995
    a = tokens_of(cfg, 600)
    b = [(a[0] + 1) % cfg["vocab"]] + a[1:]
    ra, rb = (oracle.forward(cfg, W, t)[-20:] for t in (a, b))
    assert rel_err(ra, rb) > 50 * TOL
    for toks, ref in ((a, ra), (b, rb)):
        got = run_cut(make_engine(cfg, W), toks, [500, 64, 1])
        assert rel_err(got[-20:], ref) < TOL


@pytest.mark.parametrize("name", ["mixed", "full", "recurrent"])
def test_unequal_requests_in_one_batch(name):
    """Portions beside single tokens, requests that pause, end and make way:
    every logit as if the request were alone, on a pool that only just holds
    the live ones."""
    cfg, W = make(name)
    lens = [130, 3, 61, 1, 97, 40]
    seqs = [tokens_of(cfg, n, seed=i) for i, n in enumerate(lens)]
    refs = [oracle.forward(cfg, W, s) for s in seqs]
    eng = make_engine(cfg, W, kv_blocks=23, max_batch=3)
    g = torch.Generator().manual_seed(5)
    waiting, live = list(range(len(seqs))), {}
    used, owners = set(), {}
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
            assert rel_err(logits[row:row + n], refs[i][at:at + n]) < 2 * TOL
            row += n
            live[i][1] = at + n
            used |= set(r.blocks)
            owners.setdefault(r.slot, set()).add(i)
            if at + n == len(seqs[i]):
                eng.close_request(r)
                del live[i]
    assert len(owners) == 3 and max(len(o) for o in owners.values()) > 1
    assert len(eng.allocator.free) == eng.allocator.num_blocks
    assert sorted(eng.free_slots) == [0, 1, 2]


def test_stale_pages_and_slots_do_not_leak():
    cfg, W = make("full")
    eng = make_engine(cfg, W, kv_blocks=12)
    toks = tokens_of(cfg, 100, seed=8)
    ref = oracle.forward(cfg, W, toks)
    for c in eng.caches:
        c.fill_(50.0)
    assert rel_err(run_cut(eng, toks, [7, 1, 40]), ref) < TOL
    assert rel_err(run_cut(eng, toks, [50]), ref) < TOL


def test_every_pass_has_a_cache_of_its_own():
    cfg, W = make("mixed")
    eng = make_engine(cfg, W)
    assert [i for i, _ in eng.model.runs] == [0, 1, 2, 3, 1, 2, 3, 4]
    assert [e for _, e in eng.model.runs] == [None, 0, None, None, 1, None,
                                              None, None]
    assert len({c.data_ptr() for c in eng.caches}) == 8
    # state slots for the running requests and one for padded rows
    assert eng.caches[1].shape == (7, 3, 24, 16)
    assert eng.caches[1].dtype == torch.float32
    # a cached row: key, and the rotated dimensions once more
    assert eng.caches[0].shape == (128, 2, 16, 16 + 8 + 16)
    assert eng.caches[2].shape == (128, 4, 16, 16 + 16)


def test_cache_is_bounded_by_the_window():
    cfg, W = make("mixed")
    eng = make_engine(cfg, W)
    r = eng.open_request()
    run_cut(eng, tokens_of(cfg, 400), [50, 1, 1], req=r)
    assert r.dropped > 250 and len(r.blocks) * 16 <= 64 + 50 + 32
    cfg, W = make("full")
    full = make_engine(cfg, W)
    r = full.open_request()
    run_cut(full, tokens_of(cfg, 200), [64], req=r)
    assert r.dropped == 0
    cfg, W = make("recurrent")             # nothing is cached at all
    rec = make_engine(cfg, W)
    r = rec.open_request()
    run_cut(rec, tokens_of(cfg, 100), [9], req=r)
    assert len(r.blocks) <= 2


def test_pool_slot_and_length_limits_are_errors():
    cfg, W = make("full")
    eng = make_engine(cfg, W, kv_blocks=4)
    with pytest.raises(RuntimeError, match="exhausted"):
        run_cut(eng, tokens_of(cfg, 80), [80])
    eng.cfg.max_seq_len = 20
    with pytest.raises(ValueError, match="max_seq_len"):
        run_cut(eng, tokens_of(cfg, 30), [30])
    eng = make_engine(cfg, W, max_batch=2)
    reqs = [eng.open_request() for _ in range(3)]
    eng.run_portions([(r, [1, 2], []) for r in reqs[:2]])
    with pytest.raises(RuntimeError, match="no state slot"):
        eng.run_portions([(reqs[2], [1, 2], [])])
    eng.close_request(reqs[0])
    eng.run_portions([(reqs[2], [1, 2], [])])


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
    out = eng.generate(prompt, max_new_tokens=200)
    ref = oracle.forward(cfg, W, prompt + out).argmax(-1).tolist()
    assert ref[29:-1] == out


@pytest.mark.parametrize("chunk,blocks", [(2048, 128), (20, 128), (33, 40),
                                          (16, 24), (200, 13)])
def test_scheduler_batches(chunk, blocks):
    """Admission, prompt portions beside decoding, preemption on a small
    pool: the greedy continuation never changes."""
    cfg, W = make("full")
    eng = make_engine(cfg, W, kv_blocks=blocks, max_batch=3)
    assert not eng.prefix_cache_enabled    # blocks alone are not the state
    eng.prefill_chunk = chunk
    base = tokens_of(cfg, 100, seed=4)
    prompts = [base[:n] for n in (1, 60, 100, 33, 100, 17)] + \
        [tokens_of(cfg, 70, seed=9)]
    reqs = [eng.submit(p, max_new_tokens=30) for p in prompts]
    steps = 0
    while eng.has_work():
        eng.step()
        steps += 1
        assert steps < 2000
    for r, p in zip(reqs, prompts):
        _assert_greedy(cfg, W, r, p, 30)
    if blocks == 13:
        assert eng.stats["preemptions"] > 0
    assert len(eng.allocator.free) == eng.allocator.num_blocks
    assert sorted(eng.free_slots) == [0, 1, 2]


def test_scheduler_cancel_stop_and_sampling():
    cfg, W = make("mixed")
    eng = make_engine(cfg, W)
    a = eng.submit(tokens_of(cfg, 20), max_new_tokens=50)
    first = make_engine(cfg, W).generate(tokens_of(cfg, 40), 9)
    b = eng.submit(tokens_of(cfg, 40), max_new_tokens=50,
                   stop_token_ids=(first[4],))
    c = eng.submit(tokens_of(cfg, 15), max_new_tokens=6, temperature=0.8,
                   seed=3, logprobs=2)
    for _ in range(4):
        eng.step()
    eng.cancel(a.request_id)
    while eng.has_work():
        eng.step()
    assert a.finished and len(a.output_ids) < 10
    assert b.output_ids == first[:first.index(first[4]) + 1]
    assert len(c.output_ids) == 6 and len(c.logprob_data) == 6
    assert sorted(eng.free_slots) == list(range(6))


def test_failed_step_releases_blocks_and_slots():
    cfg, W = make("mixed")
    eng = make_engine(cfg, W)
    eng.submit(tokens_of(cfg, 20))

    def boom(*_):
        raise RuntimeError("injected")
    eng.forward_plan, keep = boom, eng.forward_plan
    with pytest.raises(RuntimeError, match="injected"):
        eng.step()
    assert len(eng.allocator.free) == eng.allocator.num_blocks
    assert sorted(eng.free_slots) == list(range(6))
    eng.forward_plan = keep
    assert len(eng.generate(tokens_of(cfg, 5), 3)) == 3


# --- configuration, weights, command line -------------------------------------

def test_checkpoint_directory_round_trip(tmp_path):
    cfg, W = make("mixed")
    d = write_checkpoint(tmp_path / "m", cfg, W)
    mc = config_from_dir(d)
    back = config_from_keralorn(config_to_keralorn(mc))
    assert back.layers == mc.layers and back.loop == mc.loop
    assert mc.sliding_window == 64 and mc.norm_eps == 2e-5
    assert mc.kernel_groups == ("core", "lightning", "shared_kv")
    assert config_from_keralorn(make("full")[0]).sliding_window is None
    m = build_model(mc, dtype=torch.float32)
    load_pretrained(m, d)
    ref = load(cfg, W, torch.float32)
    for (k, a), (_, b) in zip(m.state_dict().items(),
                              ref.state_dict().items()):
        assert torch.equal(a, b), k
    del W["l2.norm1.b"]
    with pytest.raises(KeyError):
        load_pretrained(build_model(mc, dtype=torch.float32),
                        write_checkpoint(tmp_path / "bad", cfg, W))


def test_configuration_errors():
    cfg, _ = make("mixed")

    def broken(f):
        c = json.loads(json.dumps(cfg))
        f(c)
        return c
    mixer = lambda c, i: c["layers"][i]["mixer"]  # noqa: E731
    for f in (lambda c: c["layers"][0].update(type="other"),
              lambda c: c["layers"][0]["mlp"].update(kind="sparse"),
              lambda c: mixer(c, 0).update(kv_heads=4),
              lambda c: mixer(c, 0).update(vdim=19),
              lambda c: mixer(c, 0)["rot"].update(dims=22),
              lambda c: mixer(c, 0)["rot"].update(dims=3),
              lambda c: mixer(c, 0)["mask"].update(size=0),
              lambda c: mixer(c, 1).update(decay=[0.5, 0.5]),
              lambda c: mixer(c, 1).update(decay=[0.5, 0.5, 1.5]),
              lambda c: c["loop"].update(stop=6),
              lambda c: c["loop"].update(start=4),
              lambda c: c["loop"].update(times=0),
              lambda c: c.update(architecture="Other")):
        with pytest.raises(ValueError):
            c = broken(f)
            if c["architecture"] == "Other":
                from runbooks_amd.models.load import config_from_hf_json
                import tempfile
                with tempfile.NamedTemporaryFile("w", suffix=".json") as fh:
                    json.dump(c, fh)
                    fh.flush()
                    config_from_hf_json(fh.name)
            config_from_keralorn(c)
    for where in (lambda c: c, lambda c: mixer(c, 0), lambda c: c["loop"],
                  lambda c: mixer(c, 0)["rot"]["scaling"]):
        c = broken(lambda c: where(c).update(extra=1))
        with pytest.warns(UserWarning, match="without effect"):
            config_from_keralorn(c)


def test_registry_and_packing_keep_parameters():
    mc = get_config("tiny-keralorn")
    m = build_model(mc, dtype=torch.float32)
    before = {k: v.clone() for k, v in m.state_dict().items()}
    for blk in m.blocks:
        blk.fuse()
    for k, v in m.state_dict().items():
        assert torch.equal(v, before[k]), k
    assert mc.params_b > 0
    # 2 passes over layers 1 and 2: one attention run more than layers
    per_token = 2 * (16 + 24)
    assert m.kv_bytes_per_block() == 2 * per_token * 16 * 4
    assert m.state_bytes() == 4 * 4 * 3 * 16 * 24
    assert get_config("llama2-7b").kernel_groups == ("core", "main")


def test_parts_serve_another_design():
    """RMS norms, no loop, an attention layer without rotation or window:
    the same blocks under another description."""
    spec = SharedKVAttentionSpec(heads=2, kv_heads=1, dim=8, scale=0.3,
                                 rope_dims=0)
    mc = layered_config("p", [LayerSpec(spec, GLUSpec(12)),
                              LayerSpec(LightningSpec(1, 4, 4, (0.9,)), None)],
                        16, 20, max_seq_len=64)
    assert mc.norm == "rmsnorm" and mc.sliding_window is None
    eng = Engine(build_model(mc, dtype=torch.float32), device="cpu",
                 kv_blocks=16)
    toks = [3, 1, 4, 1, 5, 9, 2, 6]
    whole = run_cut(eng, toks, [8])
    assert torch.allclose(whole, run_cut(eng, toks, [1]), atol=1e-5)
    P = dict(eng.model.named_parameters())
    g = {k: v.detach().double() for k, v in P.items()}
    x = g["embed.weight"][toks]
    h = oracle.rms_norm(x, g["blocks.0.norm1.weight"], mc.norm_eps)
    W = {"a." + n: g[f"blocks.0.mixer.{n}_proj.weight"] for n in "qko"}
    m = {"heads": 2, "kv_heads": 1, "dim": 8, "scale": 0.3,
         "rot": {"base": 1e4, "dims": 0}}
    x = x + oracle.shared_kv_attention(h, W, "a.", m)
    h = oracle.rms_norm(x, g["blocks.0.norm2.weight"], mc.norm_eps)
    x = x + oracle.gated_gelu(h, *(g[f"blocks.0.mlp.{n}_proj.weight"]
                                   for n in ("gate", "up", "down")))
    h = oracle.rms_norm(x, g["blocks.1.norm1.weight"], mc.norm_eps)
    W = {"b." + n: g[f"blocks.1.mixer.{n}_proj.weight"] for n in "qkvgo"}
    W["b.norm"] = g["blocks.1.mixer.norm.weight"]
    x = x + oracle.lightning(h, W, "b.", {"heads": 1, "dim": 4, "vdim": 4,
                                          "decay": [0.9]}, mc.norm_eps)
    ref = oracle.rms_norm(x, g["norm_f.weight"], mc.norm_eps) @ \
        g["lm_head.weight"].T
    assert rel_err(whole, ref) < TOL
    with pytest.raises(ValueError, match="layout"):
        layered_config("q", [LayerSpec(spec, None),
                             get_config("tiny-pimazen").layers[0]], 16, 20)
    with pytest.raises(ValueError, match="share latents"):
        layered_config("r", get_config("tiny-pimazen").layers, 64, 20,
                       loop=LoopSpec(0, 2, 2))


def test_synthetic_model_loads_and_serves(tmp_path):
    from runbooks_amd.workloads.model_loader import materialize_synthetic
    materialize_synthetic("tiny-keralorn", tmp_path)
    mc = config_from_dir(tmp_path)
    m = load_pretrained(build_model(mc, dtype=torch.float32, seed=5),
                        tmp_path)
    out = Engine(m, device="cpu", kv_blocks=32).generate([1, 2, 3], 5)
    assert len(out) == 5


def test_http_server_serves_the_family():
    from fastapi.testclient import TestClient
    from runbooks_amd.serve import ByteTokenizer
    from runbooks_amd.serve.http import build_app
    eng = Engine("tiny-keralorn", device="cpu", dtype=torch.float32,
                 kv_blocks=64)
    with TestClient(build_app(eng, ByteTokenizer(),
                              model_name="tiny-keralorn")) as client:
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


def test_plan_flattens():
    ps = portions((3, 20, 16), (1, 0, 0), (40, 5, 0))
    ps[0].want = [0, 2]
    back = StepPlan.unflatten(StepPlan(ps).flatten())
    assert back.portions == ps
    assert {p.slot for p in back.portions} == {0, 1, 2}
    b = StepPlan(ps).build(16, [], "cpu")
    # short portions come first, with their slots
    assert b.n_short == 2 and b.n_seqs == 3 and b.max_q_long == 40
    assert b.state_slots.tolist() == [p.slot for p in ps]
