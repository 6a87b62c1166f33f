"""The Dopilorn family under tensor parallelism (gloo, 2 ranks): heads and
their states, biases, convolutions and feed-forward columns sharded, PolyNorm's
sums over all ranks; ragged steps followed by the worker rank."""
import os

import torch
import torch.distributed as dist
import torch.multiprocessing as mp

import dopilorn_oracle as oracle

PORT = 29841
LAYERS = [oracle.diff(4, 2, 12, 10, 19, mlp=oracle.dense(24)),
          oracle.delta(4, 12, mlp=oracle.dense(20)),
          oracle.latent(2, 8, 12, 20, 16),
          oracle.delta(2, 8)]


def _rank(rank, world):
    os.environ.update(MASTER_ADDR="127.0.0.1", MASTER_PORT=str(PORT),
                      RANK=str(rank), WORLD_SIZE=str(world))
    dist.init_process_group("gloo", rank=rank, world_size=world)
    try:
        from dopilorn_helpers import rel_err, run_cut, tokens_of
        from runbooks_amd.models import build_model
        from runbooks_amd.models.load import (config_from_dopilorn,
                                              convert_hf_state_dict,
                                              shard_state_dict)
        from runbooks_amd.serve import Engine
        from runbooks_amd.serve.tp_worker import (broadcast_shutdown,
                                                  worker_loop)
        cfg = oracle.make_config(LAYERS, 32, 60, (1, 3, 2))
        W = oracle.make_weights(cfg, gain=0.8)
        mc = config_from_dopilorn(cfg, {k: v.shape for k, v in W.items()})
        mc.max_seq_len = 512
        model = build_model(mc, dtype=torch.float32, tp=world)
        state = {k: v.float()
                 for k, v in convert_hf_state_dict(W, mc).items()}
        model.load_state_dict(shard_state_dict(state, model, rank, world),
                              strict=False)
        diff, delta, latent = (b.mixer for b in model.blocks[:3])
        assert diff.q_proj.weight.shape[0] == 4 * 2 * 12 // world
        assert diff.k_conv.shape[0] == 2 * 2 * 12 // world
        assert diff.v_proj.bias.shape[0] == 2 * 10 // world
        assert delta.w0.shape[0] == delta.norm.weight.shape[0] == 48 // world
        assert latent.g_proj.weight.shape[0] == 2 // world
        assert latent.dkv_proj.weight.shape[0] == 16
        eng = Engine(model, device="cpu", kv_blocks=32, max_batch=3)
        if rank:
            worker_loop(eng)
            return
        toks = tokens_of(cfg, 70)
        ref = oracle.forward(cfg, W, toks)
        assert rel_err(run_cut(eng, toks, [40, 1, 3, 17, 1]), ref) < 3e-5
        reqs = [eng.submit(toks[:n], max_new_tokens=8) for n in (5, 50, 70)]
        while eng.has_work():
            eng.step()
        for r in reqs:
            ids = r.prompt_ids + r.output_ids
            best = oracle.forward(cfg, W, ids).argmax(-1).tolist()
            n = len(r.prompt_ids)
            assert best[n - 1:-1] == ids[n:]
        broadcast_shutdown(torch.device("cpu"))
    finally:
        dist.destroy_process_group()


def test_two_ranks():
    ctx = mp.get_context("spawn")
    procs = [ctx.Process(target=_rank, args=(r, 2)) for r in range(2)]
    for p in procs:
        p.start()
    for p in procs:
        p.join(120)
    for p in procs:
        assert p.exitcode == 0
