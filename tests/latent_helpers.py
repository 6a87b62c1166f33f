"""Small latent-attention models for the tests, and ways to run them."""
import json

import torch

import latent_oracle as oracle
from runbooks_amd.models import build_model
from runbooks_amd.models.load import config_from_pimazen, convert_hf_state_dict
from runbooks_amd.serve import Engine

# layers that differ in every size, share latents over unequal windows and
# heads, and have an MLP or none
MIXED = [
    dict(heads=3, dim=20, rot_dim=12, vdim=16, kv_rank=36, window=21,
         base=500.0, ff=50, limit=1.3),
    dict(heads=2, dim=16, rot_dim=12, vdim=24, kv_rank=36, window=35,
         base=500.0, ff=None, kv_from=0, scale=0.3),
    dict(heads=1, dim=8, rot_dim=4, vdim=10, kv_rank=24, window=5,
         base=90000.0, ff=40, limit=0.8),
    dict(heads=5, dim=24, rot_dim=4, vdim=12, kv_rank=24, window=64,
         base=90000.0, ff=72, limit=2.5, kv_from=2),
]
# one layer without a window: nothing may be dropped from the cache
FULL = [
    dict(heads=2, dim=16, rot_dim=8, vdim=8, kv_rank=16, window=9, ff=32,
         limit=1.0),
    dict(heads=4, dim=8, rot_dim=16, vdim=16, kv_rank=40, window=None,
         ff=48, limit=1.5),
]
# sizes of 1: a window of the token itself, one head, one MLP unit
ONES = [
    dict(heads=1, dim=1, rot_dim=2, vdim=1, kv_rank=1, window=1, ff=1,
         limit=0.5),
    dict(heads=2, dim=3, rot_dim=2, vdim=5, kv_rank=7, window=2, ff=9,
         limit=0.5),
]
WIDE = [  # sizes of a real layer's heads, few of them
    dict(heads=9, dim=128, rot_dim=64, vdim=128, kv_rank=512, window=130,
         ff=160, limit=3.0),
    dict(heads=40, dim=64, rot_dim=32, vdim=96, kv_rank=200, window=48,
         ff=None),
]
MODELS = {"mixed": (MIXED, 48, 90), "full": (FULL, 40, 70),
          "ones": (ONES, 24, 33), "wide": (WIDE, 96, 120)}


def make(name, seed=0):
    layers, width, vocab = MODELS[name]
    cfg = oracle.make_config(layers, width, vocab, eps=2e-5)
    return cfg, oracle.make_weights(cfg, seed)


def load(cfg, W, dtype, device="cpu", tp=1):
    mc = config_from_pimazen(cfg)
    mc.max_seq_len = 2048
    model = build_model(mc, dtype=dtype, tp=tp)
    state = {k: v.to(dtype) for k, v in convert_hf_state_dict(W, mc).items()}
    missing, unexpected = model.load_state_dict(state, strict=False)
    assert not missing and not unexpected, (missing, unexpected)
    return model.to(device)


def make_engine(cfg, W, dtype=torch.float32, device="cpu", **kw):
    kw.setdefault("kv_blocks", 128)
    kw.setdefault("prefix_cache", False)
    return Engine(load(cfg, W, dtype, device), device=device, **kw)


def tokens_of(cfg, n, seed=0):
    g = torch.Generator().manual_seed(seed)
    return torch.randint(0, cfg["vocab"], (n,), generator=g).tolist()


def run_cut(eng, toks, cuts, req=None):
    """Feed one request in portions; logits at every position."""
    r = req or eng.open_request()
    out, at, i = [], 0, 0
    while at < len(toks):
        n = min(cuts[i % len(cuts)], len(toks) - at)
        out.append(eng.run_portions(
            [(r, toks[at:at + n], range(n))]).float().cpu())
        at, i = at + n, i + 1
    if req is None:
        eng.close_request(r)
    return torch.cat(out)


def rel_err(got, ref):
    """Worst row: rms of the difference over the rms of all logits."""
    d = (got.double() - ref.double()).pow(2).mean(-1).sqrt()
    return float(d.max() / ref.double().pow(2).mean().sqrt())


def close(got, ref, dtype, slack=1.0):
    """Engine logits against the oracle: 32-bit to rounding; bf16 to a mean
    error, with room for single rows that small models amplify (a gate near
    its clamp, two keys of nearly equal score)."""
    d = (got.double() - ref.double()).pow(2).mean(-1).sqrt() / \
        ref.double().pow(2).mean().sqrt()
    if dtype == torch.float32:
        return float(d.max()) < 2e-5 * slack
    return float(d.mean()) < 0.02 * slack and float(d.max()) < 0.15 * slack


def write_checkpoint(path, cfg, W):
    from safetensors.torch import save_file
    path.mkdir(parents=True, exist_ok=True)
    save_file({k: v.contiguous() for k, v in W.items()},
              str(path / "model.safetensors"))
    (path / "config.json").write_text(json.dumps(cfg))
    return path
