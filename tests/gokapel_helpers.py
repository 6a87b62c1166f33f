"""Small models of the Gokapel family for the tests, and ways to run them."""
import copy

import torch

import gokapel_oracle as oracle
from gokapel_oracle import delta, dense, moe, twin
from keralorn_helpers import portions  # noqa: F401
from latent_helpers import (rel_err, run_cut, tokens_of,  # noqa: F401
                            write_checkpoint)
from runbooks_amd.models import build_model
from runbooks_amd.models.load import (config_from_gokapel,
                                      convert_hf_state_dict)
from runbooks_amd.serve import Engine

# every size differs between layers; both mixers with every feed-forward and
# with none; one layer's weights used twice
MIXED = [delta(4, 2, 20, 12, taps=3, mlp=moe(24, 12, 3, (4, 2), 40)),
         twin(6, 2, 20, 28, 21, 12, 36, base=500.0, mlp=dense(50)),
         delta(3, 3, 12, 40, taps=5),
         delta(4, 2, 20, 12, taps=3, mlp=moe(24, 12, 3, (4, 2), 40),
               weights_of=0),
         twin(4, 4, 16, 8, 35, 6, 20, base=90000.0, scale=0.4,
              scales=(0.3, 1.2), mlp=moe(40, 6, 2, None, 24))]
# no chunks: nothing may be dropped from the cache
FULL = [twin(4, 2, 24, 16, None, 24, 40, mlp=moe(16, 8, 2, (2, 1))),
        delta(2, 1, 16, 24, mlp=dense(32)),
        twin(4, 2, 24, 16, None, 24, 40, mlp=moe(16, 8, 2, (2, 1)),
             weights_of=0)]
# sizes of 1: one head, one tap, chunks of one token, one expert, one stream
ONES = [twin(1, 1, 3, 1, 1, 2, 1, scales=(1.0, 1.0), mlp=dense(1)),
        delta(1, 1, 2, 1, taps=1, mlp=moe(1, 1, 1, (1, 1), 1)),
        delta(2, 1, 1, 3, taps=2)]
RECURRENT = [delta(4, 4, 16, 32, mlp=dense(30)),
             delta(6, 2, 40, 8, taps=2, mlp=moe(20, 10, 4, (5, 3)))]
WIDE = [delta(4, 2, 128, 128, mlp=moe(64, 16, 4, (8, 3), 96)),
        twin(8, 2, 128, 64, 130, 32, 200, base=500000.0, mlp=dense(160)),
        delta(2, 2, 64, 96, mlp=dense(100)),
        twin(3, 3, 64, 128, 48, 64, 72)]
BIG = [twin(2, 1, 256, 192, 70, 96, 24, mlp=dense(64)),
       delta(1, 1, 256, 72), delta(2, 1, 136, 264)]
# name: (layers, width, vocab, streams)
MODELS = {"mixed": (MIXED, 48, 90, 3), "full": (FULL, 40, 70, 2),
          "ones": (ONES, 24, 33, 1), "recurrent": (RECURRENT, 36, 50, 4),
          "wide": (WIDE, 96, 120, 4), "big": (BIG, 64, 60, 5)}


def make(name, seed=0):
    layers, width, vocab, streams = MODELS[name]
    cfg = oracle.make_config(copy.deepcopy(layers), width, vocab, streams,
                             mult=0.8, eps=2e-5)
    return cfg, oracle.make_weights(cfg, seed, gain=0.8)


def load(cfg, W, dtype, device="cpu", tp=1):
    mc = config_from_gokapel(cfg, {k: tuple(v.shape) for k, v in W.items()})
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
    error. Rounding may decide a few tokens of such small models (experts of
    nearly equal choice score, a unit vector or a head's result of a length
    near zero), so single rows may differ."""
    d = (got.double() - ref.double()).pow(2).mean(-1).sqrt() / \
        ref.double().pow(2).mean().sqrt()
    if dtype == torch.float32:
        return float(d.max()) < 2e-5 * slack
    return float(d.mean()) < 0.02 * slack and \
        float((d > 0.15).double().mean()) < 0.03 * slack
