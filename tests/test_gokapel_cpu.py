"""The Gokapel family on the CPU path: every op and whole engine runs against
the plain oracle (tests/gokapel_oracle.py)."""
import io
import json
import os

import numpy as np
import pytest
import torch

import gokapel_oracle as oracle
from gokapel_helpers import (MODELS, load, make, make_engine, portions,
                             rel_err, run_cut, tokens_of, write_checkpoint)
from runbooks_amd import ops
from runbooks_amd.models import build_model, get_config
from runbooks_amd.models.config import (AttentionSpec, GatedDeltaSpec,
                                        LayerSpec, MinGRUSpec, MoESpec,
                                        SquaredReluSpec, TwinSpec,
                                        layered_config)
from runbooks_amd.models.load import (config_from_dir, config_from_gokapel,
                                      config_to_gokapel, load_pretrained)
from runbooks_amd.models.ragged import StepPlan
from runbooks_amd.ops import delta as DR
from runbooks_amd.ops import min_gru as MG
from runbooks_amd.ops import moe as ME
from runbooks_amd.ops import qkv as QK
from runbooks_amd.ops import shared_kv as SK
from runbooks_amd.ops import streams as ST
from runbooks_amd.serve import Engine

TOL = 3e-5


def shapes_of(W):
    return {k: tuple(v.shape) for k, v in W.items()}


def generator(seed=0):
    g = torch.Generator().manual_seed(seed)
    return lambda *n: torch.randn(*n, generator=g)


# --- single mechanisms -------------------------------------------------------

@pytest.mark.parametrize("s", [1, 2, 5])
def test_streams_and_dynamic_tanh(s):
    """A pending result enters the streams, in all its parts; the next
    sublayer reads the new ones."""
    T, D = 6, 20
    r = generator(s)
    x, inp, mix, out = r(T, s, D), r(s), r(s, s), r(s)
    scale, bias, gate, delta, extra = r(D), r(D), r(T, D), r(3, T, D), r(T, D)
    norm = ops.DynamicTanh(D)
    for p in norm.parameters():
        p.data.copy_(r(*p.shape, 1)[..., 0])
    y = (delta.sum(0) + extra).double() * scale * torch.sigmoid(gate + bias)
    want = oracle.spread(x.double(), y, mix, out, 0.7)
    u = (want * inp[None, :, None]).sum(1)
    ref = oracle.dynamic_tanh(u, norm.weight, norm.bias, norm.alpha)
    pending = ops.Pending(delta, extra, torch.cat([r(T, 4), gate], 1), 4,
                          ST.pack_join(scale, bias, out, mix, 0.7))
    h = ops.streams_norm(x, pending, inp, norm.packed(), torch.float32)
    assert torch.allclose(x.double(), want, atol=1e-5)
    assert torch.allclose(h[:, :D].double(), ref, atol=1e-5)
    assert h.shape[1] == 32 and not h[:, D:].any()
    again = ops.streams_norm(x, None, inp, norm.packed(), torch.float32)
    assert torch.equal(again, h)


def test_squared_relu():
    y = torch.tensor([[-2.0, 0.0, 3.0, 0.5] * 8])
    assert torch.equal(ops.squared_relu(y, 16)[0, :4],
                       torch.tensor([0.0, 0.0, 9.0, 0.25]))


@pytest.mark.parametrize("dims", [0, 2, 6, 20])
def test_norm_and_rotation_of_queries_and_keys(dims):
    H, G, d, e, D, T = 4, 2, 20, 12, 24, 70
    r = generator(1)
    lay = QK.QKVLayout(H, G, d, e, dims)
    wq, wk, wv, x = r(H * d, D), r(G * d, D), r(G * e, D), r(T, D)
    norms = r(2, d)
    p = portions((T, 0, 0), blocks=9)
    b = StepPlan(p).build(16, [], "cpu", expand=False)
    y = x @ QK.pack_qkv(lay, wq, wk, wv).T
    cos, sin = ops.rope_tables(dims, 128, 300.0)
    cache = SK.alloc_shared_kv_cache(9, lay, "cpu", torch.float32)
    QK.qkv_prep(y, lay, cos, sin, b.positions, b.slots, cache, norms, 1e-3)
    rot = {"base": 300.0, "dims": dims}
    x = x.double()

    def ref(w, n, weight):
        h = oracle.rms((x @ w.double().T).view(T, n, d), 1e-3) * weight
        return oracle.rotate_pairs(h, rot)

    got = y[:, :lay.off_k].view(T, H, lay.hc)
    assert torch.allclose(got[..., :d].double(), ref(wq, H, norms[0]),
                          atol=2e-5)
    rows = cache[p[0].blocks].transpose(1, 2).reshape(-1, G, lay.ec)[:T]
    assert torch.allclose(rows[..., :d].double(), ref(wk, G, norms[1]),
                          atol=2e-5)
    assert torch.allclose(rows[..., lay.voff:lay.voff + e].double(),
                          (x @ wv.double().T).view(T, G, e), atol=1e-5)


@pytest.mark.parametrize("chunk", [None, 1, 7, 16, 33])
@pytest.mark.parametrize("cut", [0, 5, 32, 33])
def test_chunked_attention_with_a_sink(chunk, cut):
    """The last tokens of a sequence against the whole sequence's attention;
    pages before their chunk may be gone."""
    H, G, d, e, T = 4, 2, 12, 8, 80
    r = generator(3)
    lay = QK.QKVLayout(H, G, d, e, 0)
    q, k, v, sink = r(T, H, d), r(T, G, d), r(T, G, e), 2 * r(H)
    s = torch.einsum("qhd,khd->hqk", q, k.repeat_interleave(2, 1)) * 0.5
    s = s.masked_fill(~oracle.chunk_mask(T, chunk), float("-inf"))
    ref = torch.einsum("hqk,khe->qhe", oracle.sink_softmax(s, sink),
                       v.repeat_interleave(2, 1)) * 0.6
    first = cut - cut % chunk if chunk else 0
    dropped = first // 16 * 16
    p = portions((T - cut, cut, dropped), blocks=12)
    cache = torch.full((12, G, 16, lay.ec), 9.0)
    for t in range(dropped, T):
        at = t - dropped
        row = cache[p[0].blocks[at // 16], :, at % 16]
        row[:, :] = 0
        row[:, :d], row[:, lay.voff:lay.voff + e] = k[t], v[t]
    y = torch.zeros(T - cut, 128)
    y[:, :lay.off_k].view(-1, H, lay.hc)[..., :d] = q[cut:]
    b = StepPlan(p).build(16, [], "cpu")
    z = torch.zeros(T - cut, lay.n_z)
    kw = dict(chunk=chunk, sink=sink, out_scale=0.6)
    if b.n_short:
        SK.shared_kv_attend(y, lay, cache, b, 0.5, None, z, **kw)
    else:
        SK.shared_kv_flash(y, lay, cache, b, 0.5, None, z, **kw)
    assert torch.allclose(z.view(-1, H, lay.vc)[..., :e], ref[cut:],
                          atol=2e-5)


@pytest.mark.parametrize("taps,H,G,d,e", [(4, 4, 2, 12, 10), (1, 2, 2, 3, 5),
                                          (6, 3, 1, 8, 16)])
def test_delta_rule(taps, H, G, d, e):
    """Projections as given: convolution, unit vectors, decays, recurrence
    and output, in portions of several sizes."""
    D, T, ra, rg = 24, 50, 5, 7
    r = generator(taps)
    p = "m."
    W = {"m.q": r(G * d, D), "m.k": r(G * d, D), "m.v": r(H * e, D),
         "m.b": r(H, D), "m.a1": r(ra, D) / 5, "m.a2": r(H * d, ra),
         "m.g1": r(rg, D), "m.g2": r(H * e, rg), "m.norm": r(e),
         "m.A_log": r(H) - 1, "m.dt_bias": r(H * d) - 1,
         "m.o": torch.eye(H * e)}
    for n, c in (("q", G * d), ("k", G * d), ("v", H * e)):
        W[f"m.{n}.conv"] = r(c, taps)
    W = {k: v * (0.3 if v.dim() == 2 and "conv" not in k and k != "m.o"
                 else 1) for k, v in W.items()}
    x = r(T, D)
    m = {"heads": H, "kv_heads": G, "dim": d, "vdim": e}
    ref = oracle.channel_delta(x.double(), {k: v.double() for k, v in
                                            W.items()}, p, m, 1e-4)
    lay = DR.DeltaLayout(H, G, d, e, taps, ra, rg)
    y = x @ DR.pack_in(lay, *(W[p + n] for n in
                              ("q", "k", "v", "b", "a1", "g1"))).T
    y2 = y[:, lay.off_r:lay.n_y] @ DR.pack_second(lay, W["m.a2"],
                                                  W["m.g2"]).T
    conv = DR.pack_conv(lay, *(W[f"m.{n}.conv"] for n in "qkv"))
    decay = DR.pack_decay(lay, W["m.A_log"], W["m.dt_bias"])
    w = torch.nn.functional.pad(W["m.norm"], (0, lay.vc - e))
    for cuts in ([T], [1], [2, 33, 3]):
        state = DR.alloc_delta_state(2, lay, "cpu", torch.float32)
        for s in state:
            s.fill_(5.0)                   # a stale slot
        at, i, out = 0, 0, []
        while at < T:
            n = min(cuts[i % len(cuts)], T - at)
            b = StepPlan(portions((n, at, 0))).build(16, [], "cpu")
            b.state_slots[:] = 1
            o = torch.zeros(n, lay.n_o)
            a, a2 = y[at:at + n], y2[at:at + n]
            step = DR.delta_step if b.n_short else DR.delta_chunk
            step(a, a2, lay, conv, decay, state, b, o)
            z = torch.ones(n, lay.n_o + 8)
            DR.delta_out(o, lay, w, a2, z, 1e-4, None, a, state[1], b)
            assert not z[:, lay.n_o:].any()
            out.append(z[:, :lay.n_o].view(n, H, lay.vc)[..., :e])
            at, i = at + n, i + 1
        assert torch.allclose(torch.cat(out).reshape(T, -1).double(), ref,
                              atol=3e-5)
        assert (state[0][0] == 5).all() and (state[1][0] == 5).all()


def test_min_gru():
    D, R, T = 20, 12, 45
    r = generator(2)
    W = {"r.z": r(R, D), "r.z.b": r(R), "r.x": r(R, D), "r.x.b": r(R),
         "r.g": r(R, D), "r.o": torch.eye(R)}
    x = r(T, D) / 4
    ref = oracle.min_gru(x, W, "r.") * 0.4
    wide = [torch.nn.functional.pad(W["r." + n], (0, 0, 0, 4)) for n in "zxg"]
    y = torch.cat([torch.ones(T, 8)] + [x @ w.T for w in wide], 1)
    bias = torch.stack([torch.nn.functional.pad(W[f"r.{n}.b"], (0, 4))
                        for n in "zx"])
    for cuts in ([T], [1], [2, 20]):
        state, at, i, out = torch.full((2, 16), 3.0), 0, 0, []
        while at < T:
            n = min(cuts[i % len(cuts)], T - at)
            b = StepPlan(portions((n, at, 0))).build(16, [], "cpu")
            z = torch.zeros(n, 24)
            MG.min_gru(y[at:at + n], 8, bias, state, b, z, 8, 0.4)
            out.append(z[:, 8:8 + R])
            at, i = at + n, i + 1
        assert torch.allclose(torch.cat(out), ref, atol=1e-5)
        assert (state[1] == 3).all()


@pytest.mark.parametrize("E,top,groups", [(12, 3, (4, 2)), (8, 2, None),
                                          (6, 6, (3, 3)), (10, 1, (5, 1)),
                                          (1, 1, (1, 1))])
def test_routing_and_experts(E, top, groups):
    r = generator(E)
    D, F, T = 32, 16, 25
    h, z, bias = r(T, D), r(T, E), 0.3 * r(E) - 0.4
    count, keep = groups or (1, 1)
    plan = ME.moe_route(z, bias, top, count, keep)
    router = {"experts": E, "top": top}
    if groups:
        router["groups"] = {"count": count, "keep": keep}
    W = {}
    for e in range(E):
        W[f"e{e}.up"], W[f"e{e}.down"] = r(F, D) / 6, r(D, F)
    up = torch.stack([W[f"e{e}.up"] for e in range(E)])
    down = torch.stack([W[f"e{e}.down"] for e in range(E)])
    parts = ME.moe_down(ME.moe_up(h, up, plan), down, plan)
    assert parts.shape == (top, T, D)
    for t in range(T):
        picked, weights = oracle.choose(z[t], bias, router)
        assert plan.chosen[t].tolist() == picked
        assert torch.allclose(plan.weights[t], torch.stack(weights))
        ref = sum(w * oracle.squared_relu(h[t], W, f"e{e}.")
                  for e, w in zip(picked, weights))
        assert torch.allclose(parts[:, t].sum(0), ref, atol=1e-4)


def test_groups_hide_experts_whose_choices_are_negative():
    """A group that is not kept has choice scores above those of the kept
    one: hidden means minus infinity, not zero."""
    z = torch.tensor([[5.0, 0.0, 4.0, 4.0]])
    bias = torch.tensor([-0.4, -5.0, -0.9, -0.9])
    plan = ME.moe_route(z, bias, 2, 2, 1)
    assert plan.chosen.tolist() == [[0, 1]]
    s = torch.softmax(z, -1)[0]
    assert torch.allclose(plan.weights[0], s[[0, 1]])


# --- whole models -------------------------------------------------------------

@pytest.mark.parametrize("name", list(MODELS))
@pytest.mark.parametrize("cuts", [[1000], [1], [2], [3, 40, 2, 1, 17],
                                  [33, 1]])
def test_any_cut_of_the_prompt(name, cuts):
    cfg, W = make(name)
    toks = tokens_of(cfg, 60 if name in ("wide", "big") else 90)
    ref = oracle.forward(cfg, W, toks)
    eng = make_engine(cfg, W)
    assert rel_err(run_cut(eng, toks, cuts), ref) < TOL
    assert len(eng.allocator.free) == eng.allocator.num_blocks
    assert sorted(eng.free_slots) == list(range(eng.max_batch))


def test_bf16_runs_both_forms_of_every_mixer():
    """bf16 on the CPU takes the long-portion forms, too."""
    cfg, W = make("recurrent")
    toks = tokens_of(cfg, 100)
    ref = oracle.forward(cfg, W, toks)
    eng = make_engine(cfg, W, torch.bfloat16)
    assert all(b.expandable for b in eng.model.blocks)
    for cuts in ([1000], [1, 40, 20, 33]):
        d = (run_cut(eng, toks, cuts) - ref).pow(2).mean(-1).sqrt()
        assert d.mean() < 0.02 * ref.pow(2).mean().sqrt()


def test_streams_after_every_layer_run():
    cfg, W = make("mixed")
    toks = tokens_of(cfg, 70)
    want, got = [], []
    oracle.forward(cfg, W, toks, layers_out=want)
    eng = make_engine(cfg, W)
    D = cfg["width"]
    ones, none = torch.ones(cfg["streams"]), torch.zeros(2 * D + 1)
    for blk in eng.model.blocks:
        def spy(x, pending, *a, _step=blk.step):
            out = _step(x, pending, *a)
            full = x.clone()
            ops.streams_norm(full, out, ones, none, torch.float32)
            got.append(full.sum(1))
            return out
        blk.step = spy
    run_cut(eng, toks, [1000])
    assert len(got) == len(want) == 5
    for g, w in zip(got, want):
        assert (g.double() - w).abs().max() < 1e-4


def _left(c, i):
    return c["layers"][i]["mixer"]["left"]


def _both(c, f):
    for i in (0, 3):
        f(c["layers"][i]["mlp"])


CHANGES = {
    "chunk 1 up": lambda c: _left(c, 1)["mask"].update(size=22),
    "chunk 1 down": lambda c: _left(c, 1)["mask"].update(size=20),
    "chunk 4 up": lambda c: _left(c, 4)["mask"].update(size=36),
    "no chunk": lambda c: _left(c, 4).pop("mask"),
    "scale": lambda c: _left(c, 4).update(scale=0.41),
    "base": lambda c: _left(c, 1)["rot"].update(base=510.0),
    "rotated dims": lambda c: _left(c, 4)["rot"].update(dims=8),
    "left scale": lambda c: c["layers"][1]["mixer"].update(left_scale=0.72),
    "right scale": lambda c: c["layers"][4]["mixer"].update(right_scale=1.1),
    "eps": lambda c: c["norm"].update(eps=2e-3),
    "residual": lambda c: c.update(residual_mult=0.81),
    "embedding": lambda c: c["embedding"].update(scale=3.1),
    "top": lambda c: _both(c, lambda m: m["router"].update(top=2)),
    "kept groups": lambda c: _both(
        c, lambda m: m["router"]["groups"].update(keep=3)),
    "group size": lambda c: _both(
        c, lambda m: m["router"]["groups"].update(count=2)),
    "no groups": lambda c: _both(c, lambda m: m["router"].pop("groups")),
    "no shared expert": lambda c: _both(c, lambda m: m.pop("shared")),
    "no feed-forward": lambda c: c["layers"][1].update(mlp=None),
    "whose weights": lambda c: c["layers"].insert(
        2, c["layers"].pop(3)),
}


@pytest.mark.parametrize("change", list(CHANGES))
def test_every_constant_is_read(change):
    """Each constant, and each chunk by one token, shows in the oracle far
    beyond the tolerance that the engine keeps."""
    cfg, W = make("mixed")
    toks = tokens_of(cfg, 90)
    ref = oracle.forward(cfg, W, toks)
    if change == "whose weights":          # layers 2 and 3 in turn
        W = {("l3" + k[2:] if k.startswith("l2.") else k): v
             for k, v in W.items()}
    CHANGES[change](cfg)
    moved = oracle.forward(cfg, W, toks)
    assert rel_err(moved, ref) > 30 * TOL
    drop = {"no shared expert": ("l0.mlp.shared",),
            "no feed-forward": ("l1.mlp", "l1.norm2", "l1.hc2", "l1.rg2",
                                "l1.ls2")}.get(change, ())
    W = {k: v for k, v in W.items() if not k.startswith(tuple(drop))} \
        if drop else W
    assert rel_err(run_cut(make_engine(cfg, W), toks, [25]), moved) < 3 * TOL


@pytest.mark.parametrize("name", [
    "l0.norm1.b", "l2.norm1.alpha", "final.norm.b", "l1.ls1", "l0.ls2",
    "l1.rg1.b", "l4.rg2", "l0.hc1.in", "l1.hc2.out", "l2.hc1.mix",
    "l0.mix.A_log", "l0.mix.dt_bias", "l2.mix.norm", "l2.mix.k.conv",
    "l1.mix.left.sink", "l1.mix.left.k.norm", "l4.mix.right.z.b",
    "l0.mlp.correction"])
def test_every_tensor_counts(name):
    cfg, W = make("mixed")
    toks = tokens_of(cfg, 40)
    ref = oracle.forward(cfg, W, toks)
    W[name] = (W[name].float() * 0.5 - 0.2).flip(-1).to(W[name].dtype) \
        if W[name].dim() else W[name] * 0.5
    moved = oracle.forward(cfg, W, toks)
    assert rel_err(moved, ref) > 50 * TOL
    assert rel_err(run_cut(make_engine(cfg, W), toks, [25]), moved) < 3 * TOL


def test_mixing_is_indexed_from_to():
    cfg, W = make("mixed")
    toks = tokens_of(cfg, 30)
    ref = oracle.forward(cfg, W, toks)
    W["l1.hc1.mix"] = W["l1.hc1.mix"].T.contiguous()
    moved = oracle.forward(cfg, W, toks)
    assert rel_err(moved, ref) > 50 * TOL
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
    """One early token changes logits far behind it, through a state or the
    attention without chunks, and the engine follows."""
    cfg, W = make(name)
    for k in W:
        if k.endswith(("A_log", "z.b")):   # states that forget slowly
            W[k] = W[k] - (5 if k.endswith("A_log") else 3)
    a = tokens_of(cfg, 300)
    b = [(a[0] + 1) % cfg["vocab"]] + a[1:]
    ra, rb = (oracle.forward(cfg, W, t)[-20:] for t in (a, b))
    assert rel_err(ra, rb) > 30 * TOL
    for toks, ref in ((a, ra), (b, rb)):
        got = run_cut(make_engine(cfg, W), toks, [200, 64, 1])
        assert rel_err(got[-20:], ref) < TOL


@pytest.mark.parametrize("name", ["mixed", "full", "recurrent"])
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
    cfg, W = make("full")
    eng = make_engine(cfg, W, kv_blocks=12)
    toks = tokens_of(cfg, 100, seed=8)
    ref = oracle.forward(cfg, W, toks)
    for t in _tensors(eng.caches):
        t.fill_(50.0)
    assert rel_err(run_cut(eng, toks, [7, 1, 40]), ref) < TOL
    assert rel_err(run_cut(eng, toks, [50]), ref) < TOL


def test_every_layer_has_a_cache_of_its_own():
    """Also one that uses another's weights."""
    cfg, W = make("mixed")
    eng = make_engine(cfg, W)
    assert [i for i, _ in eng.model.runs] == [0, 1, 2, 0, 4]
    assert len(eng.model.blocks) == 4
    tensors = _tensors(eng.caches)
    assert len({t.data_ptr() for t in tensors}) == len(tensors) == 10
    # state slots for the running requests and one for padded rows
    S, tails = eng.caches[0]
    assert S.shape == (7, 4, 24, 16) and S.dtype == torch.float32
    assert tails.shape == (7, 2, 2 * 2 * 24 + 4 * 16)
    kv, state = eng.caches[1]
    assert kv.shape == (128, 2, 16, 24 + 32)
    assert state.shape == (7, 40) and state.dtype == torch.float32
    per_slot = sum(t[0].numel() * t.element_size() for t in tensors
                   if t.shape[0] == 7)
    assert eng.model.state_bytes() == per_slot


def test_cache_is_bounded_by_the_chunk():
    cfg, W = make("mixed")
    eng = make_engine(cfg, W)
    r = eng.open_request()
    run_cut(eng, tokens_of(cfg, 300), [50, 1, 1], req=r)
    assert r.dropped > 220 and len(r.blocks) * 16 <= 35 + 50 + 32
    cfg, W = make("full")
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
    cfg, W = make("full")
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
    back = config_from_gokapel(config_to_gokapel(mc), shapes_of(W))
    assert back.layers == mc.layers and back.streams == mc.streams == 3
    assert (back.residual_mult, back.embed_scale) == (0.8, 3.0)
    assert mc.layers[0].mixer.decay_rank == 6      # from the tensors
    assert mc.layers[0].mixer.gate_rank == 10
    assert mc.sliding_window == 35 and mc.norm_eps == 2e-5
    assert mc.kernel_groups == ("core", "delta", "shared_kv",
                                "streams")
    m = build_model(mc, dtype=torch.float32)
    load_pretrained(m, d)
    ref = load(cfg, W, torch.float32)
    for (k, a), (_, b) in zip(m.state_dict().items(),
                              ref.state_dict().items()):
        assert torch.equal(a, b), k
    del W["l2.hc1.mix"]
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
    layer = lambda c, i: c["layers"][i]  # noqa: E731
    for f in (lambda c: layer(c, 0).update(type="other"),
              lambda c: layer(c, 1)["mlp"].update(kind="sparse"),
              lambda c: layer(c, 0)["mixer"].update(kv_heads=3),
              lambda c: _left(c, 1).update(kv_heads=4),
              lambda c: _left(c, 1)["rot"].update(dims=22),
              lambda c: _left(c, 1)["rot"].update(dims=3),
              lambda c: _left(c, 1)["mask"].update(size=0),
              lambda c: layer(c, 0)["mlp"]["router"].update(top=7),
              lambda c: layer(c, 0)["mlp"]["router"]["groups"].update(count=5),
              lambda c: layer(c, 0)["mlp"]["router"]["groups"].update(keep=5),
              lambda c: layer(c, 3).update(weights_of=1),
              lambda c: layer(c, 3).update(weights_of=9),
              lambda c: layer(c, 3).update(weights_of=3),
              lambda c: c.update(streams=0)):
        with pytest.raises(ValueError):
            config_from_gokapel(broken(f), shapes)
    with pytest.raises(ValueError, match="no tensor"):
        config_from_gokapel(cfg, {})
    for where in (lambda c: c, lambda c: layer(c, 0)["mixer"],
                  lambda c: _left(c, 1)["rot"],
                  lambda c: layer(c, 0)["mlp"]["router"]):
        c = broken(lambda c: where(c).update(extra=1))
        with pytest.warns(UserWarning, match="without effect"):
            config_from_gokapel(c, shapes)


def test_registry_and_packing_keep_parameters():
    mc = get_config("tiny-gokapel")
    m = build_model(mc, dtype=torch.float32)
    before = {k: v.clone() for k, v in m.state_dict().items()}
    for blk in m.blocks:
        blk.fuse()
    for k, v in m.state_dict().items():
        assert torch.equal(v, before[k]), k
    assert mc.params_b > 0 and len(m.blocks) == 4
    # two attention layers of two heads
    assert m.kv_bytes_per_block() == 2 * 2 * (24 + 16) * 16 * 4


def test_parts_serve_another_design():
    """One stream that passes its sum on, no chunk, no rotation, one expert:
    the same blocks under another description."""
    left = AttentionSpec(heads=2, kv_heads=1, dim=8, vdim=4, scale=0.3,
                         rope_dims=0)
    mc = layered_config(
        "p", [LayerSpec(TwinSpec(left, MinGRUSpec(5)), SquaredReluSpec(12)),
              LayerSpec(GatedDeltaSpec(2, 1, 4, 4, 2, 3, 3),
                        MoESpec(ff=6, experts=2, top=1))],
        16, 20, max_seq_len=64, norm="dyt", streams=1)
    eng = Engine(mc, dtype=torch.float32, device="cpu", kv_blocks=16)
    toks = [3, 1, 4, 1, 5, 9, 2, 6]
    whole = run_cut(eng, toks, [8])
    assert torch.allclose(whole, run_cut(eng, toks, [1]), atol=1e-5)
    with pytest.raises(ValueError, match="layout"):
        layered_config("q", [LayerSpec(TwinSpec(left, MinGRUSpec(5)), None)],
                       16, 20)
    with pytest.raises(ValueError, match="mlp"):
        layered_config("r", [LayerSpec(TwinSpec(left, MinGRUSpec(5)),
                                       get_config("tiny-keralorn").layers[0]
                                       .mlp)],
                       16, 20, norm="dyt", streams=2)


def test_synthetic_model_loads_and_serves(tmp_path):
    from runbooks_amd.workloads.model_loader import materialize_synthetic
    materialize_synthetic("tiny-gokapel", tmp_path)
    mc = config_from_dir(tmp_path)
    m = load_pretrained(build_model(mc, dtype=torch.float32, seed=5),
                        tmp_path)
    out = Engine(m, device="cpu", kv_blocks=32).generate([1, 2, 3], 5)
    assert len(out) == 5


def test_http_server_serves_the_family():
    from fastapi.testclient import TestClient
    from runbooks_amd.serve import ByteTokenizer
    from runbooks_amd.serve.http import build_app
    eng = Engine("tiny-gokapel", device="cpu", dtype=torch.float32,
                 kv_blocks=64)
    with TestClient(build_app(eng, ByteTokenizer(),
                              model_name="tiny-gokapel")) as client:
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
