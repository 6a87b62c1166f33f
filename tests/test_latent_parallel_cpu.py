"""Latent attention under tensor parallelism (gloo, 2 ranks): heads and MLP
columns sharded, the latent cache replicated, ragged steps followed by the
worker rank."""
import os

import torch
import torch.distributed as dist
import torch.multiprocessing as mp

import latent_oracle as oracle

PORT = 29817
LAYERS = [dict(heads=4, dim=12, rot_dim=8, vdim=10, kv_rank=20, window=19,
               ff=24, limit=1.1),
          dict(heads=2, dim=8, rot_dim=8, vdim=16, kv_rank=20, window=40,
               ff=None, kv_from=0)]


def _rank(rank, world):
    os.environ.update(MASTER_ADDR="127.0.0.1", MASTER_PORT=str(PORT),
                      RANK=str(rank), WORLD_SIZE=str(world))
    dist.init_process_group("gloo", rank=rank, world_size=world)
    try:
        from latent_helpers import rel_err, run_cut, tokens_of
        from runbooks_amd.models import build_model
        from runbooks_amd.models.load import (config_from_pimazen,
                                              convert_hf_state_dict,
                                              shard_state_dict)
        from runbooks_amd.serve import Engine
        from runbooks_amd.serve.tp_worker import (broadcast_shutdown,
                                                  worker_loop)
        cfg = oracle.make_config(LAYERS, 32, 60)
        W = oracle.make_weights(cfg)
        mc = config_from_pimazen(cfg)
        mc.max_seq_len = 512
        model = build_model(mc, dtype=torch.float32, tp=world)
        state = {k: v.float()
                 for k, v in convert_hf_state_dict(W, mc).items()}
        model.load_state_dict(shard_state_dict(state, model, rank, world),
                              strict=False)
        assert model.blocks[0].attn.q_proj.weight.shape[0] == 4 * 20 // world
        eng = Engine(model, device="cpu", kv_blocks=32)
        if rank:
            worker_loop(eng)
            return
        toks = tokens_of(cfg, 90)
        ref = oracle.forward(cfg, W, toks)
        assert rel_err(run_cut(eng, toks, [40, 1, 3, 17, 1]), ref) < 2e-5
        reqs = [eng.submit(toks[:n], max_new_tokens=12) for n in (5, 50, 90)]
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
