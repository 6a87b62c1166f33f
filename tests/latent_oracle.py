"""Plain, slow reference of the Pimazen design, written from its equations.

One function per mechanism, whole sequences only, no cache, no batching,
nothing shared with the product path. Weights come as a dict of tensors
under the design's own names ('l0.mix.q', ...), the configuration as the
parsed config.json. Everything runs in the dtype the caller gives
(float64 by default), so it serves as the numerics oracle of the tests.
"""
from __future__ import annotations

import math

import torch


def rms_norm(x, w, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * w


def rotate_interleaved(x, positions, base, dims):
    """x [T, ..., d]: pairs (2i, 2i+1) of the first `dims` dimensions turn
    by position * base^(-2i/dims); later dimensions pass."""
    out = x.clone()
    for i in range(dims // 2):
        ang = positions.to(x.dtype) * float(base) ** (-2.0 * i / dims)
        c, s = torch.cos(ang), torch.sin(ang)
        while c.dim() < x.dim() - 1:
            c, s = c[..., None], s[..., None]
        u, v = x[..., 2 * i], x[..., 2 * i + 1]
        out[..., 2 * i] = u * c - v * s
        out[..., 2 * i + 1] = v * c + u * s
    return out


def latent_and_key(h, w_dkv, w_norm, eps, kv_rank, rot, positions):
    """The cached pair: normed latent c [T, kv_rank] and the rotated key
    part [T, rot_dim] that all heads share."""
    d = h @ w_dkv.T
    c = rms_norm(d[:, :kv_rank], w_norm, eps)
    return c, rotate_interleaved(d[:, kv_rank:], positions, rot["base"],
                                 rot["dims"])


def window_mask(T, size):
    """[T, T] bool: query i sees key j iff 0 <= i - j < size (size None:
    every earlier key)."""
    i = torch.arange(T)
    dist = i[:, None] - i[None, :]
    ok = dist >= 0
    return ok if size is None else ok & (dist < size)


def softmax_attention(q, k, v, scale, mask):
    """q, k [T, H, d], v [T, H, e] -> [T, H, e]."""
    out = torch.zeros(q.shape[0], q.shape[1], v.shape[2], dtype=q.dtype)
    for h in range(q.shape[1]):
        s = (q[:, h] @ k[:, h].T) * scale
        s = s.masked_fill(~mask, -math.inf)
        s = s - s.max(dim=-1, keepdim=True).values
        p = torch.exp(s)
        out[:, h] = (p / p.sum(-1, keepdim=True)) @ v[:, h]
    return out


def latent_attention(h, W, pre, m, eps, positions, latents, idx):
    """One mixer on its normed input; `latents` maps a layer index to the
    (c, rotated key) that layer computed."""
    H, dim, rd, vd = m["heads"], m["dim"], m["rot_dim"], m["vdim"]
    T = h.shape[0]
    q = (h @ W[pre + "q"].T).reshape(T, H, dim + rd)
    q_un = q[..., :dim]
    q_rot = rotate_interleaved(q[..., dim:], positions, m["rot"]["base"],
                               m["rot"]["dims"])
    if m.get("kv_from") is None:
        latents[idx] = latent_and_key(h, W[pre + "dkv"], W[pre + "dkv.norm"],
                                      eps, m["kv_rank"], m["rot"], positions)
        src = idx
    else:
        src = m["kv_from"]
    c, k_rot = latents[src]
    k_un = (c @ W[pre + "uk"].T).reshape(T, H, dim)
    v = (c @ W[pre + "uv"].T).reshape(T, H, vd)
    k = torch.cat([k_un, k_rot[:, None].expand(T, H, rd)], dim=-1)
    q = torch.cat([q_un, q_rot], dim=-1)
    size = (m.get("mask") or {}).get("size")
    o = softmax_attention(q, k, v, m["scale"], window_mask(T, size))
    o = o.reshape(T, H * vd) * torch.sigmoid(h @ W[pre + "g"].T)
    return o @ W[pre + "o"].T


def clamped_glu(h, w_gate, w_up, w_down, limit, alpha=1.702, shift=1.0):
    g = torch.clamp(h @ w_gate.T, max=limit)
    u = torch.clamp(h @ w_up.T, min=-limit, max=limit)
    return (g * torch.sigmoid(alpha * g) * (u + shift)) @ w_down.T


def forward(cfg, W, tokens, dtype=torch.float64, layers_out=None):
    """Logits [T, vocab] of one sequence; `layers_out` collects the
    residual after every layer."""
    W = {k: (v.to(dtype) if v.is_floating_point() else v)
         for k, v in W.items()}
    eps = cfg["norm"]["eps"]
    tokens = torch.as_tensor(tokens, dtype=torch.long)
    positions = torch.arange(len(tokens))
    x = W["embed"][tokens]
    latents = {}
    for i, lay in enumerate(cfg["layers"]):
        h = rms_norm(x, W[f"l{i}.norm1"], eps)
        y = latent_attention(h, W, f"l{i}.mix.", lay["mixer"], eps,
                             positions, latents, i)
        mlp = lay.get("mlp")
        if mlp is not None:
            p = f"l{i}.mlp."
            y = y + clamped_glu(h, W[p + "gate"], W[p + "up"], W[p + "down"],
                                mlp["limit"])
        x = x + y
        if layers_out is not None:
            layers_out.append(x)
    return rms_norm(x, W["final.norm"], eps) @ W["head"].T


# --- small models for the tests --------------------------------------------

def make_config(layers, width, vocab, eps=1e-5):
    """`layers`: dicts with heads, dim, rot_dim, vdim, kv_rank, window,
    base, scale, kv_from, ff, limit (ff None: no feed-forward)."""
    out = []
    for s in layers:
        mixer = {"dim": s["dim"], "heads": s["heads"],
                 "kv_rank": s["kv_rank"],
                 "rot": {"base": float(s.get("base", 10000.0)),
                         "dims": s["rot_dim"]},
                 "rot_dim": s["rot_dim"],
                 "scale": s.get("scale",
                                (s["dim"] + s["rot_dim"]) ** -0.5),
                 "vdim": s["vdim"]}
        mixer["mask"] = {"size": s["window"]}
        if s.get("kv_from") is not None:
            mixer["kv_from"] = s["kv_from"]
        mlp = None if s.get("ff") is None else {
            "kind": "dense", "ff": s["ff"], "limit": s.get("limit", 7.0)}
        out.append({"type": "latent_attention", "mixer": mixer, "mlp": mlp})
    return {"architecture": "Pimazen", "layers": out, "norm": {"eps": eps},
            "vocab": vocab, "width": width}


def make_weights(cfg, seed=0, gain=1.0, dtype=torch.bfloat16):
    g = torch.Generator().manual_seed(seed)

    def lin(o, i, k=gain):
        return (torch.randn(o, i, generator=g) * k / i ** 0.5).to(dtype)

    def vec(n):
        return (1.0 + 0.3 * torch.randn(n, generator=g)).to(dtype)

    D, V = cfg["width"], cfg["vocab"]
    W = {"embed": lin(V, D, D ** 0.5), "head": lin(V, D), "final.norm": vec(D)}
    for i, lay in enumerate(cfg["layers"]):
        m = lay["mixer"]
        H, R = m["heads"], m["kv_rank"]
        W[f"l{i}.norm1"] = vec(D)
        p = f"l{i}.mix."
        W[p + "q"] = lin(H * (m["dim"] + m["rot_dim"]), D, 2 * gain)
        if m.get("kv_from") is None:
            W[p + "dkv"] = lin(R + m["rot_dim"], D, 2 * gain)
            W[p + "dkv.norm"] = vec(R)
        W[p + "uk"] = lin(H * m["dim"], R)
        W[p + "uv"] = lin(H * m["vdim"], R)
        W[p + "g"] = lin(H * m["vdim"], D)
        W[p + "o"] = lin(D, H * m["vdim"], 2 * gain)
        if lay["mlp"] is not None:
            p, F = f"l{i}.mlp.", lay["mlp"]["ff"]
            W[p + "gate"] = lin(F, D, 2 * gain)
            W[p + "up"] = lin(F, D, 2 * gain)
            W[p + "down"] = lin(D, F)
    return W
