"""Load HuggingFace-format checkpoints into the native Transformer.

The import path of the platform: the model-loader image downloads HF
weights into /content/artifacts (reference
examples/facebook-opt-125m/base-model.yaml:7-9), and the trainer/server load them from
/content/model. This module maps the llama / falcon / OPT HF naming onto
the native module tree, splits falcon's fused query_key_value, and
TP-shards each tensor for the local rank.
"""
from __future__ import annotations

import json
import warnings
from pathlib import Path

import torch

from .config import ModelConfig
from .transformer import Transformer


def detect_family(cfg: ModelConfig) -> str:
    if cfg.layers is not None:
        return {"streams": "gokapel", "dual": "dopilorn", "shared": "pimazen",
                "sequence": "keralorn"}[cfg.layout]
    if cfg.pos == "learned":
        return "gpt2" if cfg.act == "gelu_tanh" else "opt"
    if cfg.parallel_residual:
        return "falcon"
    return "llama"


# ---------------------------------------------------------------------------
# HF name -> native name
# ---------------------------------------------------------------------------

def _map_llama(name: str):
    n = name
    n = n.replace("model.embed_tokens", "embed")
    n = n.replace("model.layers.", "blocks.")
    n = n.replace(".self_attn.", ".attn.")
    n = n.replace(".input_layernorm.", ".norm1.")
    n = n.replace(".post_attention_layernorm.", ".norm2.")
    n = n.replace("model.norm", "norm_f")
    return n


def _map_opt(name: str):
    n = name
    n = n.replace("model.decoder.embed_tokens", "embed")
    n = n.replace("model.decoder.embed_positions", "embed_pos")
    n = n.replace("model.decoder.layers.", "blocks.")
    n = n.replace(".self_attn.", ".attn.")
    n = n.replace(".out_proj.", ".o_proj.")
    n = n.replace(".self_attn_layer_norm.", ".norm1.")
    n = n.replace("model.decoder.final_layer_norm", "norm_f")
    n = n.replace(".final_layer_norm.", ".norm2.")
    n = n.replace(".fc1.", ".mlp.fc1.")
    n = n.replace(".fc2.", ".mlp.down_proj.")
    return n


def _map_gpt2(name: str):
    n = name
    if not n.startswith(("transformer.", "lm_head")):
        n = "transformer." + n          # GPT2Model vs GPT2LMHeadModel
    n = n.replace("transformer.wte", "embed")
    n = n.replace("transformer.wpe", "embed_pos")
    n = n.replace("transformer.h.", "blocks.")
    n = n.replace(".attn.c_proj.", ".attn.o_proj.")
    n = n.replace(".mlp.c_fc.", ".mlp.fc1.")
    n = n.replace(".mlp.c_proj.", ".mlp.down_proj.")
    n = n.replace(".ln_1.", ".norm1.")
    n = n.replace(".ln_2.", ".norm2.")
    n = n.replace("transformer.ln_f", "norm_f")
    return n


def _map_falcon(name: str):
    n = name
    n = n.replace("transformer.word_embeddings", "embed")
    n = n.replace("transformer.h.", "blocks.")
    n = n.replace(".self_attention.dense.", ".attn.o_proj.")
    n = n.replace(".mlp.dense_h_to_4h.", ".mlp.fc1.")
    n = n.replace(".mlp.dense_4h_to_h.", ".mlp.down_proj.")
    # falcon-7b single-norm / falcon-40b two-norm naming
    n = n.replace(".input_layernorm.", ".norm1.")
    n = n.replace(".ln_attn.", ".norm1.")
    n = n.replace(".ln_mlp.", ".norm2.")
    n = n.replace("transformer.ln_f", "norm_f")
    return n


_PIMAZEN = {"mix.q": "attn.q_proj", "mix.dkv": "attn.dkv_proj",
            "mix.dkv.norm": "attn.kv_norm", "mix.uk": "attn.uk_proj",
            "mix.uv": "attn.uv_proj", "mix.g": "attn.g_proj",
            "mix.o": "attn.o_proj", "mlp.gate": "mlp.gate_proj",
            "mlp.up": "mlp.up_proj", "mlp.down": "mlp.down_proj",
            "norm1": "norm1"}
_PIMAZEN_TOP = {"embed": "embed", "final.norm": "norm_f", "head": "lm_head"}


def _map_pimazen(name: str):
    if name in _PIMAZEN_TOP:
        return _PIMAZEN_TOP[name] + ".weight"
    layer, _, rest = name.partition(".")
    if layer[:1] == "l" and layer[1:].isdigit() and rest in _PIMAZEN:
        return f"blocks.{layer[1:]}.{_PIMAZEN[rest]}.weight"
    return name


_KERALORN = {"mix.q": "mixer.q_proj", "mix.k": "mixer.k_proj",
             "mix.v": "mixer.v_proj", "mix.g": "mixer.g_proj",
             "mix.o": "mixer.o_proj", "mix.norm": "mixer.norm",
             "mlp.gate": "mlp.gate_proj", "mlp.up": "mlp.up_proj",
             "mlp.down": "mlp.down_proj", "norm1": "norm1", "norm2": "norm2"}
_KERALORN_TOP = {"embed": "embed", "final.norm": "norm_f", "head": "lm_head",
                 "loop.in": "loop_in"}


def _map_keralorn(name: str):
    base, kind = ((name[:-2], "bias") if name.endswith(".b")
                  else (name, "weight"))
    if base in _KERALORN_TOP:
        return f"{_KERALORN_TOP[base]}.{kind}"
    layer, _, rest = base.partition(".")
    if layer[:1] == "l" and layer[1:].isdigit() and rest in _KERALORN:
        return f"blocks.{layer[1:]}.{_KERALORN[rest]}.{kind}"
    return name


_GOKAPEL = {
    **{f"mix.{n}": f"mixer.{n}_proj.weight" for n in
       ("q", "k", "v", "b", "a1", "a2", "g1", "g2", "o")},
    **{f"mix.{n}.conv": f"mixer.{n}_conv" for n in ("q", "k", "v")},
    "mix.A_log": "mixer.a_log", "mix.dt_bias": "mixer.dt_bias",
    "mix.norm": "mixer.norm.weight",
    **{f"mix.left.{n}": f"mixer.left.{n}_proj.weight"
       for n in ("q", "k", "v", "o")},
    "mix.left.q.norm": "mixer.left.q_norm.weight",
    "mix.left.k.norm": "mixer.left.k_norm.weight",
    "mix.left.sink": "mixer.left.sink",
    **{f"mix.right.{n}": f"mixer.right.{n}_proj.weight"
       for n in ("z", "x", "g", "o")},
    "mix.right.z.b": "mixer.right.z_proj.bias",
    "mix.right.x.b": "mixer.right.x_proj.bias",
    "mlp.up": "mlp.up_proj.weight", "mlp.down": "mlp.down_proj.weight",
    "mlp.router": "mlp.router.weight", "mlp.correction": "mlp.correction",
    "mlp.shared.up": "mlp.shared.up_proj.weight",
    "mlp.shared.down": "mlp.shared.down_proj.weight",
    **{f"{a}{n}": f"join{n}.{b}" for n in "12" for a, b in
       (("ls", "scale"), ("rg", "gate.weight"))},
    **{f"{a}{n}.{c}": f"join{n}.{b}" for n in "12" for a, c, b in
       (("rg", "b", "gate.bias"), ("hc", "in", "inp"), ("hc", "out", "out"),
        ("hc", "mix", "mix"))}}


def _map_gokapel(name: str, cfg: ModelConfig):
    """Experts keep their numbers; blocks count the layers that have
    parameters."""
    if name == "embed":
        return "embed.weight"
    base, kind = next(((name[:-len(end)], k) for end, k in
                       ((".b", "bias"), (".alpha", "alpha"))
                       if name.endswith(end)), (name, "weight"))
    if base == "final.norm":
        return f"norm_f.{kind}"
    layer, _, rest = name.partition(".")
    if layer[:1] != "l" or not layer[1:].isdigit() or \
            int(layer[1:]) not in cfg.owners:
        return name
    block = f"blocks.{cfg.owners.index(int(layer[1:]))}."
    if rest in _GOKAPEL:
        return block + _GOKAPEL[rest]
    if base.partition(".")[2] in ("norm1", "norm2"):
        return f"{block}{base.partition('.')[2]}.{kind}"
    part = rest.split(".")
    if len(part) == 3 and part[0] == "mlp" and part[1][:1] == "e" and \
            part[1][1:].isdigit() and part[2] in ("up", "down"):
        return f"{block}mlp.experts.{part[1][1:]}.{part[2]}_proj.weight"
    return name


_DOPILORN = {
    **{f"mix.{n}": f"mixer.{n}_proj.weight" for n in
       ("q", "k", "v", "o", "r", "a", "g", "w1", "w2", "dq", "uq", "dkv",
        "uk", "uv")},
    **{f"mix.{n}.b": f"mixer.{n}_proj.bias" for n in ("q", "k", "v", "a")},
    **{f"mix.{n}.conv": f"mixer.{n}_conv" for n in ("q", "k", "v")},
    **{f"mix.{n}": f"mixer.{n}" for n in
       ("lq1", "lk1", "lq2", "lk2", "w0")},
    "mix.norm": "mixer.norm.weight", "mix.dq.norm": "mixer.q_norm.weight",
    "mix.dkv.norm": "mixer.kv_norm.weight",
    "mlp.up": "mlp.up_proj.weight", "mlp.down": "mlp.down_proj.weight",
    "mlp.act": "mlp.act",
    **{f"norm{n}": f"norm{n}.weight" for n in "12"},
    **{f"canon{n}": f"canon{n}" for n in "12"}}
_DOPILORN_TOP = {"embed": "embed.weight", "final.norm": "norm_f.weight",
                 "head": "lm_head.weight", "loop.in": "loop_in.weight",
                 "loop.step": "loop_step"}


def _map_dopilorn(name: str):
    if name in _DOPILORN_TOP:
        return _DOPILORN_TOP[name]
    layer, _, rest = name.partition(".")
    if layer[:1] == "l" and layer[1:].isdigit() and rest in _DOPILORN:
        return f"blocks.{layer[1:]}.{_DOPILORN[rest]}"
    return name


def _split_falcon_qkv(w: torch.Tensor, cfg: ModelConfig):
    """Falcon fuses QKV as [n_kv_groups, (g_q + 2), head_dim, hidden] with
    the group's q heads followed by its k and v head."""
    g = cfg.num_heads // cfg.num_kv_heads
    dh = cfg.head_dim
    w = w.view(cfg.num_kv_heads, g + 2, dh, cfg.hidden_size)
    q = w[:, :g].reshape(cfg.num_heads * dh, cfg.hidden_size)
    k = w[:, g].reshape(cfg.num_kv_heads * dh, cfg.hidden_size)
    v = w[:, g + 1].reshape(cfg.num_kv_heads * dh, cfg.hidden_size)
    return q, k, v


def convert_hf_state_dict(hf_state: dict, cfg: ModelConfig) -> dict:
    family = detect_family(cfg)
    out: dict[str, torch.Tensor] = {}
    mapper = {"llama": _map_llama, "opt": _map_opt,
              "falcon": _map_falcon, "gpt2": _map_gpt2,
              "pimazen": _map_pimazen,
              "keralorn": _map_keralorn, "dopilorn": _map_dopilorn,
              "gokapel": lambda n: _map_gokapel(n, cfg)}[family]
    for name, w in hf_state.items():
        if name.endswith(".rotary_emb.inv_freq"):
            continue
        if family == "gpt2":
            if name.endswith((".attn.bias", ".attn.masked_bias")):
                continue  # causal-mask buffers, not weights
            if ".attn.c_attn." in name:
                # Conv1D fused QKV: weight [in, 3*out] -> three [out, in]
                blk = name.split(".")[name.split(".").index("h") + 1]
                if name.endswith(".weight"):
                    qw, kw, vw = w.t().chunk(3, dim=0)
                else:
                    qw, kw, vw = w.chunk(3, dim=0)
                kind = "weight" if name.endswith(".weight") else "bias"
                out[f"blocks.{blk}.attn.q_proj.{kind}"] = qw.contiguous()
                out[f"blocks.{blk}.attn.k_proj.{kind}"] = kw.contiguous()
                out[f"blocks.{blk}.attn.v_proj.{kind}"] = vw.contiguous()
                continue
            if name.endswith(".weight") and w.dim() == 2 and any(
                    k in name for k in (".c_proj.", ".c_fc.")):
                w = w.t().contiguous()  # Conv1D stores [in, out]
        if family == "falcon" and ".self_attention.query_key_value." in name:
            blk = name.split(".")[2 if name.startswith("transformer") else 1]
            q, k, v = _split_falcon_qkv(w, cfg)
            out[f"blocks.{blk}.attn.q_proj.weight"] = q
            out[f"blocks.{blk}.attn.k_proj.weight"] = k
            out[f"blocks.{blk}.attn.v_proj.weight"] = v
            continue
        n = mapper(name)
        if family == "opt" and n.startswith("embed_pos"):
            # OPT's learned positions carry a +2 offset (HF
            # OPTLearnedPositionalEmbedding); drop the two pad rows.
            w = w[2:]
        out[n] = w
    # gemma stores RMSNorm weights zero-centered (x * (1 + w)); fold the
    # +1 at import so the fused rmsnorm kernel stays family-agnostic
    if cfg.act == "gelu_glu" and cfg.norm == "rmsnorm":
        for k in list(out):
            if k.endswith((".norm1.weight", ".norm2.weight")) or                     k == "norm_f.weight":
                out[k] = out[k].float() + 1.0
    # tied embeddings: derive lm_head when absent
    if "lm_head.weight" not in out and "embed.weight" in out:
        out["lm_head.weight"] = out["embed.weight"]
    return out


# ---------------------------------------------------------------------------
# TP sharding
# ---------------------------------------------------------------------------

def shard_state_dict(state: dict, model: Transformer, rank: int,
                     tp: int) -> dict:
    """Slice full tensors to this rank's shard, matching parallel/tp.py's
    column (output-dim) / row (input-dim) split."""
    if tp <= 1:
        return state
    out = {}
    named = dict(model.named_parameters())
    named.update(dict(model.named_buffers()))
    for k, w in state.items():
        tgt = named.get(k)
        if tgt is None or tgt.shape == w.shape:
            out[k] = w
            continue
        if tgt.shape[0] != w.shape[0]:        # column-parallel (incl. bias)
            s = tgt.shape[0]
            out[k] = w[rank * s:(rank + 1) * s]
        elif w.dim() == 2 and tgt.shape[1] != w.shape[1]:  # row-parallel
            s = tgt.shape[1]
            out[k] = w[:, rank * s:(rank + 1) * s]
        else:
            out[k] = w
    return out


# ---------------------------------------------------------------------------
# Entry points
# ---------------------------------------------------------------------------

def load_safetensors_dir(path: str | Path) -> dict:
    from safetensors.torch import load_file
    path = Path(path)
    files = sorted(path.glob("*.safetensors"))
    if not files:
        raise FileNotFoundError(f"no .safetensors under {path}")
    state: dict[str, torch.Tensor] = {}
    for f in files:
        state.update(load_file(str(f)))
    return state


def _only(obj, known, where):
    """obj, after a warning about keys that would have no effect."""
    extra = set(obj) - set(known)
    if extra:
        warnings.warn(f"{where}: keys without effect: {sorted(extra)}")
    return obj


def config_from_keralorn(d: dict, name: str = "keralorn") -> ModelConfig:
    """ModelConfig from a Keralorn config.json. A layer type or kind this
    framework does not have is an error; an unknown key is reported."""
    from .config import (GLUSpec, LayerSpec, LightningSpec, LoopSpec,
                         RopeScaling, SharedKVAttentionSpec, layered_config)

    def attention(m, where):
        _only(m, ("heads", "kv_heads", "dim", "vdim", "scale", "rot",
                  "mask"), where)
        if m.get("vdim", m["dim"]) != m["dim"]:
            raise ValueError(f"{where}: keys double as values, but vdim "
                             f"{m['vdim']} is not dim {m['dim']}")
        rot = _only(m["rot"], ("base", "dims", "scaling"), where)
        scaling = rot.get("scaling")
        if scaling is not None:
            keys = ("factor", "low", "high", "original")
            scaling = RopeScaling(*(float(_only(scaling, keys, where)[k])
                                    for k in keys))
        mask = _only(m.get("mask") or {}, ("size",), where)
        return SharedKVAttentionSpec(
            heads=m["heads"], kv_heads=m["kv_heads"], dim=m["dim"],
            scale=float(m["scale"]), rope_dims=rot["dims"],
            rope_base=float(rot["base"]), rope_scaling=scaling,
            window=mask.get("size"))

    def lightning(m, where):
        _only(m, ("heads", "dim", "vdim", "decay"), where)
        return LightningSpec(m["heads"], m["dim"], m["vdim"],
                             tuple(float(x) for x in m["decay"]))

    mixers = {"attention": attention, "lightning": lightning}
    _only(d, ("architecture", "layers", "loop", "norm", "vocab", "width",
              "max_seq_len"), "config")
    layers = []
    for i, lay in enumerate(d["layers"]):
        where = f"layer {i}"
        _only(lay, ("type", "mixer", "mlp"), where)
        if lay["type"] not in mixers:
            raise ValueError(f"{where}: type {lay['type']!r}")
        mlp = lay.get("mlp")
        if mlp is not None:
            _only(mlp, ("kind", "ff"), where)
            if mlp["kind"] != "dense":
                raise ValueError(f"{where}: mlp kind {mlp['kind']!r}")
            mlp = GLUSpec(mlp["ff"])
        layers.append(LayerSpec(mixers[lay["type"]](lay["mixer"], where),
                                mlp))
    loop = d.get("loop")
    if loop is not None:
        keys = ("start", "stop", "times")
        loop = LoopSpec(*(_only(loop, keys, "loop")[k] for k in keys))
    kw = {"max_seq_len": d["max_seq_len"]} if "max_seq_len" in d else {}
    return layered_config(name, layers, d["width"], d["vocab"],
                          norm_eps=float(_only(d["norm"], ("eps",),
                                               "norm")["eps"]),
                          norm="layernorm", loop=loop, **kw)


def config_to_keralorn(cfg: ModelConfig) -> dict:
    """The config.json of a Keralorn model (inverse of
    config_from_keralorn)."""
    from dataclasses import asdict
    layers = []
    for lay in cfg.layers:
        m = lay.mixer
        if lay.attends:
            rot = {"base": m.rope_base, "dims": m.rope_dims}
            if m.rope_scaling is not None:
                rot["scaling"] = asdict(m.rope_scaling)
            mixer = {"heads": m.heads, "kv_heads": m.kv_heads, "dim": m.dim,
                     "vdim": m.dim, "scale": m.scale, "rot": rot}
            if m.window is not None:
                mixer["mask"] = {"size": m.window}
        else:
            mixer = {"heads": m.heads, "dim": m.dim, "vdim": m.vdim,
                     "decay": list(m.decay)}
        layers.append({
            "type": "attention" if lay.attends else "lightning",
            "mixer": mixer,
            "mlp": lay.mlp and {"kind": "dense", "ff": lay.mlp.ff}})
    out = {"architecture": "Keralorn", "layers": layers,
           "norm": {"eps": cfg.norm_eps}, "vocab": cfg.vocab_size,
           "width": cfg.hidden_size, "max_seq_len": cfg.max_seq_len}
    if cfg.loop is not None:
        out["loop"] = asdict(cfg.loop)
    return out


def tensor_shapes(path: str | Path) -> dict:
    """Shapes of a checkpoint directory's tensors, from the headers."""
    from safetensors import safe_open
    shapes = {}
    for f in sorted(Path(path).glob("*.safetensors")):
        with safe_open(str(f), framework="pt") as st:
            for name in st.keys():
                shapes[name] = tuple(st.get_slice(name).get_shape())
    return shapes


def config_from_gokapel(d: dict, shapes: dict, name: str = "gokapel"
                        ) -> ModelConfig:
    """ModelConfig from a Gokapel config.json and the shapes of its tensors
    (the inner sizes of the delta mixer's decay and gate projections stand
    only there). A type or kind this framework does not have is an error; an
    unknown key is reported."""
    from .config import (AttentionSpec, GatedDeltaSpec, LayerSpec, MinGRUSpec,
                         MoESpec, SquaredReluSpec, TwinSpec, layered_config)

    def rows(i, tensor):
        seen = set()
        while i not in seen and i < len(d["layers"]) and \
                d["layers"][i].get("weights_of") is not None:
            seen.add(i)
            i = d["layers"][i]["weights_of"]
        full = f"l{i}.mix.{tensor}"
        if full not in shapes:
            raise ValueError(f"no tensor {full} to take a size from")
        return shapes[full][0]

    def delta(m, where, i):
        _only(m, ("heads", "kv_heads", "dim", "vdim", "conv"), where)
        return GatedDeltaSpec(m["heads"], m["kv_heads"], m["dim"], m["vdim"],
                              m["conv"], rows(i, "a1"), rows(i, "g1"))

    def parallel(m, where, i):
        _only(m, ("left", "right", "left_scale", "right_scale"), where)
        a = _only(m["left"], ("heads", "kv_heads", "dim", "vdim", "scale",
                              "rot", "mask"), where + " left")
        rot = _only(a["rot"], ("base", "dims"), where)
        mask = _only(a.get("mask") or {}, ("size",), where)
        right = _only(m["right"], ("width",), where + " right")
        return TwinSpec(
            AttentionSpec(a["heads"], a["kv_heads"], a["dim"], a["vdim"],
                          float(a["scale"]), rot["dims"],
                          float(rot["base"]), mask.get("size")),
            MinGRUSpec(right["width"]), float(m["left_scale"]),
            float(m["right_scale"]))

    def feed_forward(m, where):
        if m["kind"] == "dense":
            return SquaredReluSpec(_only(m, ("kind", "ff"), where)["ff"])
        if m["kind"] != "moe":
            raise ValueError(f"{where}: mlp kind {m['kind']!r}")
        _only(m, ("kind", "expert", "router", "shared"), where)
        r = _only(m["router"], ("experts", "top", "groups"), where)
        groups = _only(r.get("groups") or {"count": 1, "keep": 1},
                       ("count", "keep"), where)
        shared = _only(m.get("shared") or {}, ("ff",), where)
        return MoESpec(_only(m["expert"], ("ff",), where)["ff"],
                       r["experts"], r["top"], groups["count"],
                       groups["keep"], shared.get("ff", 0))

    mixers = {"channel_delta": delta, "parallel": parallel}
    _only(d, ("architecture", "embedding", "layers", "norm", "residual_mult",
              "streams", "vocab", "width", "max_seq_len"), "config")
    layers = []
    for i, lay in enumerate(d["layers"]):
        where = f"layer {i}"
        _only(lay, ("type", "mixer", "mlp", "weights_of"), where)
        if lay["type"] not in mixers:
            raise ValueError(f"{where}: type {lay['type']!r}")
        mlp = lay.get("mlp")
        layers.append(LayerSpec(
            mixers[lay["type"]](lay["mixer"], where, i),
            None if mlp is None else feed_forward(mlp, where),
            lay.get("weights_of")))
    kw = {"max_seq_len": d["max_seq_len"]} if "max_seq_len" in d else {}
    return layered_config(
        name, layers, d["width"], d["vocab"],
        norm_eps=float(_only(d["norm"], ("eps",), "norm")["eps"]),
        norm="dyt", tie_embeddings=True, streams=d["streams"],
        residual_mult=float(d["residual_mult"]),
        embed_scale=float(_only(d["embedding"], ("scale",),
                                "embedding")["scale"]), **kw)


def config_to_gokapel(cfg: ModelConfig) -> dict:
    """The config.json of a Gokapel model (inverse of config_from_gokapel)."""
    layers = []
    for lay in cfg.layers:
        m, f = lay.mixer, lay.mlp
        if lay.attends:
            a = m.left
            left = {"heads": a.heads, "kv_heads": a.kv_heads, "dim": a.dim,
                    "vdim": a.vdim, "scale": a.scale,
                    "rot": {"base": a.rope_base, "dims": a.rope_dims}}
            if a.chunk is not None:
                left["mask"] = {"size": a.chunk}
            mixer = {"left": left, "left_scale": m.left_scale,
                     "right": {"width": m.right.width},
                     "right_scale": m.right_scale}
        else:
            mixer = {"heads": m.heads, "kv_heads": m.kv_heads, "dim": m.dim,
                     "vdim": m.vdim, "conv": m.conv}
        mlp = None
        if f is not None and not hasattr(f, "experts"):
            mlp = {"kind": "dense", "ff": f.ff}
        elif f is not None:
            mlp = {"kind": "moe", "expert": {"ff": f.ff},
                   "router": {"experts": f.experts, "top": f.top,
                              "groups": {"count": f.groups, "keep": f.keep}}}
            if f.shared_ff:
                mlp["shared"] = {"ff": f.shared_ff}
        entry = {"type": "parallel" if lay.attends else "channel_delta",
                 "mixer": mixer, "mlp": mlp}
        if lay.weights_of is not None:
            entry["weights_of"] = lay.weights_of
        layers.append(entry)
    return {"architecture": "Gokapel",
            "embedding": {"scale": cfg.embed_scale}, "layers": layers,
            "norm": {"eps": cfg.norm_eps},
            "residual_mult": cfg.residual_mult, "streams": cfg.streams,
            "vocab": cfg.vocab_size, "width": cfg.hidden_size,
            "max_seq_len": cfg.max_seq_len}


def config_from_dopilorn(d: dict, shapes: dict, name: str = "dopilorn"
                         ) -> ModelConfig:
    """ModelConfig from a Dopilorn config.json and the shapes of its tensors
    (the inner size of the delta mixer's decay projection stands only there).
    A type or kind this framework does not have is an error; an unknown key
    is reported."""
    from .config import (DiffAttentionSpec, GeneralDeltaSpec,
                         LatentAttentionSpec, LayerSpec, LoopSpec,
                         PolyNormSpec, layered_config)

    def delta(m, where, i):
        _only(m, ("heads", "dim"), where)
        full = f"l{i}.mix.w1"
        if full not in shapes:
            raise ValueError(f"no tensor {full} to take a size from")
        return GeneralDeltaSpec(m["heads"], m["dim"], shapes[full][0])

    def attention(m, where, i):
        _only(m, ("heads", "kv_heads", "dim", "vdim", "scale", "diff", "conv",
                  "mask"), where)
        mask = _only(m.get("mask") or {}, ("size",), where)
        return DiffAttentionSpec(
            m["heads"], m["kv_heads"], m["dim"], m["vdim"],
            float(m["scale"]), float(m["diff"]), m["conv"], mask.get("size"))

    def latent(m, where, i):
        _only(m, ("heads", "dim", "vdim", "q_rank", "kv_rank", "scale"),
              where)
        return LatentAttentionSpec(
            heads=m["heads"], dim=m["dim"], rot_dim=0, vdim=m["vdim"],
            kv_rank=m["kv_rank"], scale=float(m["scale"]),
            q_rank=m["q_rank"], head_gate=True)

    mixers = {"general_delta": delta, "attention": attention,
              "latent_attention": latent}
    _only(d, ("architecture", "canon", "layers", "logit_softcap", "loop",
              "norm", "vocab", "width", "max_seq_len"), "config")
    layers = []
    for i, lay in enumerate(d["layers"]):
        where = f"layer {i}"
        _only(lay, ("type", "mixer", "mlp"), where)
        if lay["type"] not in mixers:
            raise ValueError(f"{where}: type {lay['type']!r}")
        mlp = lay.get("mlp")
        if mlp is not None:
            _only(mlp, ("kind", "ff"), where)
            if mlp["kind"] != "dense":
                raise ValueError(f"{where}: mlp kind {mlp['kind']!r}")
            mlp = PolyNormSpec(mlp["ff"])
        layers.append(LayerSpec(mixers[lay["type"]](lay["mixer"], where, i),
                                mlp))
    loop = d.get("loop")
    if loop is not None:
        keys = ("start", "stop", "times")
        loop = LoopSpec(*(_only(loop, keys, "loop")[k] for k in keys),
                        step=True)
    kw = {"max_seq_len": d["max_seq_len"]} if "max_seq_len" in d else {}
    cap = d.get("logit_softcap")
    return layered_config(
        name, layers, d["width"], d["vocab"],
        norm_eps=float(_only(d["norm"], ("eps",), "norm")["eps"]),
        norm_offset=1.0, loop=loop,
        canon=_only(d["canon"], ("taps",), "canon")["taps"],
        logit_softcap=None if cap is None else float(cap), **kw)


def config_to_dopilorn(cfg: ModelConfig) -> dict:
    """The config.json of a Dopilorn model (inverse of
    config_from_dopilorn)."""
    from .config import DiffAttentionSpec, GeneralDeltaSpec
    layers = []
    for lay in cfg.layers:
        m = lay.mixer
        if isinstance(m, GeneralDeltaSpec):
            kind, mixer = "general_delta", {"heads": m.heads, "dim": m.dim}
        elif isinstance(m, DiffAttentionSpec):
            kind = "attention"
            mixer = {"heads": m.heads, "kv_heads": m.kv_heads, "dim": m.dim,
                     "vdim": m.vdim, "scale": m.scale, "diff": m.diff,
                     "conv": m.conv}
            if m.window is not None:
                mixer["mask"] = {"size": m.window}
        else:
            kind = "latent_attention"
            mixer = {"heads": m.heads, "dim": m.dim, "vdim": m.vdim,
                     "q_rank": m.q_rank, "kv_rank": m.kv_rank,
                     "scale": m.scale}
        layers.append({"type": kind, "mixer": mixer, "mlp": lay.mlp and
                       {"kind": "dense", "ff": lay.mlp.ff}})
    out = {"architecture": "Dopilorn", "canon": {"taps": cfg.canon},
           "layers": layers, "norm": {"eps": cfg.norm_eps},
           "vocab": cfg.vocab_size, "width": cfg.hidden_size,
           "max_seq_len": cfg.max_seq_len}
    if cfg.logit_softcap is not None:
        out["logit_softcap"] = cfg.logit_softcap
    if cfg.loop is not None:
        out["loop"] = {k: getattr(cfg.loop, k)
                       for k in ("start", "stop", "times")}
    return out


def config_from_pimazen(d: dict, name: str = "pimazen") -> ModelConfig:
    """ModelConfig from a Pimazen config.json. A layer type or kind this
    framework does not have is an error; an unknown key is reported."""
    from .config import (GatedMLPSpec, LatentAttentionSpec, LayerSpec,
                         layered_config)

    only = _only
    only(d, ("architecture", "layers", "norm", "vocab", "width",
             "max_seq_len"), "config")
    layers = []
    for i, lay in enumerate(d["layers"]):
        where = f"layer {i}"
        only(lay, ("type", "mixer", "mlp"), where)
        if lay["type"] != "latent_attention":
            raise ValueError(f"{where}: type {lay['type']!r}")
        m = only(lay["mixer"], ("heads", "dim", "rot_dim", "vdim", "kv_rank",
                                "scale", "rot", "mask", "kv_from"), where)
        rot = only(m["rot"], ("base", "dims"), where)
        mask = only(m.get("mask") or {}, ("size",), where)
        mixer = LatentAttentionSpec(
            heads=m["heads"], dim=m["dim"], rot_dim=m["rot_dim"],
            vdim=m["vdim"], kv_rank=m["kv_rank"], scale=float(m["scale"]),
            rope_base=float(rot["base"]), rope_dims=rot["dims"],
            window=mask.get("size"), kv_from=m.get("kv_from"))
        mlp = lay.get("mlp")
        if mlp is not None:
            only(mlp, ("kind", "ff", "limit"), where)
            if mlp["kind"] != "dense":
                raise ValueError(f"{where}: mlp kind {mlp['kind']!r}")
            mlp = GatedMLPSpec(mlp["ff"], float(mlp["limit"]))
        layers.append(LayerSpec(mixer, mlp))
    kw = {"max_seq_len": d["max_seq_len"]} if "max_seq_len" in d else {}
    return layered_config(name, layers, d["width"], d["vocab"],
                          norm_eps=float(only(d["norm"], ("eps",),
                                              "norm")["eps"]), **kw)


def config_to_pimazen(cfg: ModelConfig) -> dict:
    """The config.json of a Pimazen model (inverse of config_from_pimazen)."""
    layers = []
    for lay in cfg.layers:
        m = lay.mixer
        mixer = {"heads": m.heads, "dim": m.dim, "rot_dim": m.rot_dim,
                 "vdim": m.vdim, "kv_rank": m.kv_rank, "scale": m.scale,
                 "rot": {"base": m.rope_base, "dims": m.rotation[1]}}
        if m.window is not None:
            mixer["mask"] = {"size": m.window}
        if m.kv_from is not None:
            mixer["kv_from"] = m.kv_from
        mlp = None if lay.mlp is None else {
            "kind": "dense", "ff": lay.mlp.ff, "limit": lay.mlp.limit}
        layers.append({"type": "latent_attention", "mixer": mixer,
                       "mlp": mlp})
    return {"architecture": "Pimazen", "layers": layers,
            "norm": {"eps": cfg.norm_eps}, "vocab": cfg.vocab_size,
            "width": cfg.hidden_size, "max_seq_len": cfg.max_seq_len}


def config_from_dir(path: str | Path, default: str | None = None
                    ) -> ModelConfig:
    """The configuration of a checkpoint directory: a registered name or
    explicit fields this framework wrote, a Pimazen, Keralorn, Gokapel or
    Dopilorn config, or an HF one; `default` names the registry entry of a
    directory that says nothing."""
    from .config import get_config, list_configs, register
    marker = Path(path) / "config.json"
    meta = json.loads(marker.read_text()) if marker.exists() else {}
    if meta.get("runbooks_amd_config") in list_configs():
        return get_config(meta["runbooks_amd_config"])
    if "runbooks_amd_fields" in meta:
        return register(ModelConfig(**meta["runbooks_amd_fields"]))
    if {"architecture", "model_type", "architectures"} & set(meta):
        return config_from_hf_json(marker)
    if default is None:
        raise ValueError(f"no model configuration in {marker}")
    return get_config(default)


def config_from_hf_json(path: str | Path) -> ModelConfig:
    """Derive a ModelConfig from an HF config.json (for models not in the
    registry)."""
    d = json.loads(Path(path).read_text())
    if "architecture" in d:
        readers = {"Pimazen": config_from_pimazen,
                   "Keralorn": config_from_keralorn,
                   "Gokapel": lambda d: config_from_gokapel(
                       d, tensor_shapes(Path(path).parent)),
                   "Dopilorn": lambda d: config_from_dopilorn(
                       d, tensor_shapes(Path(path).parent))}
        if d["architecture"] not in readers:
            raise ValueError(f"unsupported architecture {d['architecture']}")
        return readers[d["architecture"]](d)
    mt = d.get("model_type", "llama")
    if mt == "gemma":
        heads = d["num_attention_heads"]
        return ModelConfig(
            d.get("_name_or_path", "hf-gemma"),
            vocab_size=d["vocab_size"], hidden_size=d["hidden_size"],
            num_layers=d["num_hidden_layers"], num_heads=heads,
            num_kv_heads=d.get("num_key_value_heads", heads),
            intermediate_size=d["intermediate_size"],
            max_seq_len=d.get("max_position_embeddings", 8192),
            head_dim=d.get("head_dim", d["hidden_size"] // heads),
            norm_eps=d.get("rms_norm_eps", 1e-6),
            rope_theta=d.get("rope_theta", 10000.0),
            act="gelu_glu", tie_embeddings=True,
            embed_scale=d["hidden_size"] ** 0.5)
    if mt == "qwen2":
        return ModelConfig(
            d.get("_name_or_path", "hf-qwen2"),
            vocab_size=d["vocab_size"], hidden_size=d["hidden_size"],
            num_layers=d["num_hidden_layers"],
            num_heads=d["num_attention_heads"],
            num_kv_heads=d.get("num_key_value_heads",
                               d["num_attention_heads"]),
            intermediate_size=d["intermediate_size"],
            max_seq_len=d.get("max_position_embeddings", 32768),
            norm_eps=d.get("rms_norm_eps", 1e-6),
            rope_theta=d.get("rope_theta", 1000000.0),
            qkv_bias=True,
            tie_embeddings=d.get("tie_word_embeddings", False))
    if mt in ("llama", "mistral"):
        return ModelConfig(
            d.get("_name_or_path", "hf-llama"),
            vocab_size=d["vocab_size"], hidden_size=d["hidden_size"],
            num_layers=d["num_hidden_layers"],
            num_heads=d["num_attention_heads"],
            num_kv_heads=d.get("num_key_value_heads",
                               d["num_attention_heads"]),
            intermediate_size=d["intermediate_size"],
            max_seq_len=d.get("max_position_embeddings", 4096),
            norm_eps=d.get("rms_norm_eps", 1e-5),
            rope_theta=d.get("rope_theta", 10000.0))
    if mt in ("falcon", "RefinedWeb", "RefinedWebModel"):
        heads = d["num_attention_heads"]
        return ModelConfig(
            d.get("_name_or_path", "hf-falcon"),
            vocab_size=d["vocab_size"], hidden_size=d["hidden_size"],
            num_layers=d["num_hidden_layers"], num_heads=heads,
            num_kv_heads=d.get("num_kv_heads",
                               heads if not d.get("multi_query", True) else 1),
            intermediate_size=4 * d["hidden_size"],
            head_dim=d["hidden_size"] // heads,
            norm="layernorm", act="gelu", parallel_residual=True,
            tie_embeddings=True)
    if mt == "gpt2":
        return ModelConfig(
            d.get("_name_or_path", "hf-gpt2"),
            vocab_size=d["vocab_size"], hidden_size=d["n_embd"],
            num_layers=d["n_layer"], num_heads=d["n_head"],
            num_kv_heads=d["n_head"],
            intermediate_size=d.get("n_inner") or 4 * d["n_embd"],
            max_seq_len=d.get("n_positions", 1024),
            norm="layernorm", act="gelu_tanh", pos="learned",
            tie_embeddings=True, mlp_bias=True, attn_bias=True)
    if mt == "opt":
        return ModelConfig(
            d.get("_name_or_path", "hf-opt"),
            vocab_size=d["vocab_size"], hidden_size=d["hidden_size"],
            num_layers=d["num_hidden_layers"],
            num_heads=d["num_attention_heads"],
            num_kv_heads=d["num_attention_heads"],
            intermediate_size=d["ffn_dim"],
            max_seq_len=d.get("max_position_embeddings", 2048),
            norm="layernorm", act="relu", pos="learned",
            tie_embeddings=True, mlp_bias=True, attn_bias=True)
    raise ValueError(f"unsupported model_type {mt}")


def load_pretrained(model: Transformer, path: str | Path, rank: int = 0,
                    tp: int = 1, strict: bool = True) -> Transformer:
    """Load an HF-format checkpoint directory into `model` (TP-sharded)."""
    hf = load_safetensors_dir(path)
    state = convert_hf_state_dict(hf, model.cfg)
    state = shard_state_dict(state, model, rank, tp)
    state = {k: v.to(model.dtype) if v.is_floating_point() else v
             for k, v in state.items()}
    missing, unexpected = model.load_state_dict(state, strict=False)
    unexpected = [u for u in unexpected if "rotary" not in u]
    missing = [m for m in missing if not m.startswith("rope_")]
    if strict and (missing or unexpected):
        raise KeyError(f"load_pretrained: missing={missing[:5]} "
                       f"unexpected={unexpected[:5]}")
    return model
