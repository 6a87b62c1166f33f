"""Small models of the Dopilorn family for the tests, and ways to run them."""
import copy

import torch

import dopilorn_oracle as oracle
from dopilorn_oracle import delta, dense, diff, latent
from keralorn_helpers import portions  # noqa: F401
from latent_helpers import (rel_err, run_cut, tokens_of,  # noqa: F401
                            write_checkpoint)
from runbooks_amd.models import build_model
from runbooks_amd.models.load import (config_from_dopilorn,
                                      convert_hf_state_dict)
from runbooks_amd.serve import Engine

# every size differs between layers; every mixer with and without a
# feed-forward; a loop over two layers
MIXED = [diff(6, 2, 20, 28, 21, taps=2, diff=0.3, mlp=dense(50)),
         delta(3, 20),
         latent(5, 12, 20, 28, 36, mlp=dense(72)),
         diff(4, 4, 16, 8, 35, taps=5, diff=0.7, scale=0.4),
         delta(2, 12, mlp=dense(40)),
         latent(2, 24, 10, 20, 44, scale=0.3)]
# only windows: the cache is bounded
WINDOWS = [diff(2, 1, 12, 20, 9, mlp=dense(32)), delta(4, 8),
           diff(4, 2, 24, 8, 26, taps=4, mlp=dense(24))]
# sizes of 1: one head, a window of the token itself, one tap, one pass
ONES = [diff(1, 1, 1, 1, 1, taps=1, scale=1.0, mlp=dense(1)),
        delta(1, 1, mlp=dense(1)), latent(1, 1, 1, 1, 1),
        diff(2, 1, 3, 5, 2, taps=2), delta(2, 3, mlp=dense(9))]
RECURRENT = [delta(2, 24, mlp=dense(30)), delta(5, 8)]
WIDE = [diff(4, 2, 64, 128, 130, mlp=dense(160)),
        latent(9, 128, 96, 96, 200, mlp=dense(96)), delta(3, 128),
        diff(3, 3, 48, 48, 48, taps=4), delta(2, 64, mlp=dense(100)),
        latent(3, 64, 128, 40, 512)]
BIG = [diff(2, 1, 128, 256, 70, mlp=dense(64)), delta(1, 256),
       latent(2, 200, 256, 264, 72), diff(1, 1, 192, 64, 40), delta(2, 136)]
# name: (layers, width, vocab, loop, taps of the input convolution, cap)
MODELS = {"mixed": (MIXED, 48, 90, (1, 4, 2), 4, 20.0),
          "windows": (WINDOWS, 40, 70, None, 3, None),
          "ones": (ONES, 24, 33, (0, 5, 1), 1, 5.0),
          "recurrent": (RECURRENT, 36, 50, (0, 1, 3), 6, 50.0),
          "wide": (WIDE, 96, 120, (3, 5, 2), 4, 30.0),
          "big": (BIG, 64, 60, None, 2, 10.0)}


def make(name, seed=0):
    layers, width, vocab, loop, taps, cap = MODELS[name]
    cfg = oracle.make_config(copy.deepcopy(layers), width, vocab, loop, taps,
                             cap, eps=2e-5)
    return cfg, oracle.make_weights(cfg, seed, gain=0.8)


def load(cfg, W, dtype, device="cpu", tp=1):
    mc = config_from_dopilorn(cfg, {k: tuple(v.shape) for k, v in W.items()})
    mc.max_seq_len = 2048
    model = build_model(mc, dtype=dtype, tp=tp)
    state = {k: v.to(dtype) for k, v in convert_hf_state_dict(W, mc).items()}
    missing, unexpected = model.load_state_dict(state, strict=False)
    assert not missing and not unexpected, (missing, unexpected)
    return model.to(device)


def make_engine(cfg, W, dtype=torch.float32, device="cpu", **kw):
    kw.setdefault("kv_blocks", 128)
    kw.setdefault("max_batch", 6)
    return Engine(load(cfg, W, dtype, device), device=device, **kw)


def close(got, ref, dtype, slack=1.0):
    """Engine logits against the oracle: 32-bit to rounding; bf16 to a mean
    error. A head's difference of two maps, or a head's result, may have a
    length near zero in such small models, so single rows may differ."""
    d = (got.double() - ref.double()).pow(2).mean(-1).sqrt() / \
        ref.double().pow(2).mean().sqrt()
    if dtype == torch.float32:
        return float(d.max()) < 3e-5 * slack
    return float(d.mean()) < 0.025 * slack and \
        float((d > 0.15).double().mean()) < 0.03 * slack
