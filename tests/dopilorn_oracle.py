"""Plain, slow reference of the Dopilorn design, written from its equations.

One function per mechanism, whole sequences only, no cache, no batching,
nothing shared with the product path. Weights come as a dict of tensors
under the design's own names ('l0.mix.q', ...), the configuration as the
parsed config.json. Everything runs in the dtype the caller gives (float64
by default), so it serves as the numerics oracle of the tests.
"""
from __future__ import annotations

import math

import torch


def rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def centered_norm(x, w, eps):
    """RMS norm whose weight is stored around zero."""
    return rms(x, eps) * (1 + w)


def causal_conv(x, w):
    """Causal convolution of every channel: x [T, n], w [n, taps]; the last
    column of w belongs to the current token."""
    taps = w.shape[1]
    out = torch.zeros_like(x)
    for t in range(x.shape[0]):
        for j in range(taps):
            src = t - (taps - 1) + j
            if src >= 0:
                out[t] = out[t] + x[src] * w[:, j]
    return out


def canon(h, w):
    return h + causal_conv(h, w)


# --- generalized delta rule ---------------------------------------------------

def delta_recurrence(r, k, v, w, a):
    """All [T, H, d] (v [T, H, e]) -> [T, H, e]."""
    T, H, d = k.shape
    S = torch.zeros(H, d, v.shape[2], dtype=k.dtype)
    out = torch.zeros_like(v)
    for t in range(T):
        u = k[t] / torch.sqrt((k[t] * k[t]).sum(-1, keepdim=True) + 1e-6)
        seen = (u[:, :, None] * S).sum(1)                    # u^T S, [H, e]
        S = w[t][:, :, None] * S \
            - (a[t] * u)[:, :, None] * seen[:, None, :] \
            + k[t][:, :, None] * v[t][:, None, :]
        out[t] = (S * r[t][:, :, None]).sum(1)
    return out


def channel_decay(h, W, p):
    z = torch.tanh(h @ W[p + "w1"].T) @ W[p + "w2"].T + W[p + "w0"]
    return torch.exp(-math.exp(-0.5) * torch.sigmoid(z))


def general_delta(h, W, p, m, eps):
    T, H, d = h.shape[0], m["heads"], m["dim"]

    def heads(x):
        return x.reshape(T, H, d)

    r, k, v = (heads(h @ W[p + n].T) for n in "rkv")
    a = heads(torch.sigmoid(h @ W[p + "a"].T + W[p + "a.b"]))
    o = delta_recurrence(r, k, v, heads(channel_decay(h, W, p)), a)
    o = rms(o, eps).reshape(T, H * d) * W[p + "norm"]
    return (o * torch.sigmoid(h @ W[p + "g"].T)) @ W[p + "o"].T


# --- differential attention ---------------------------------------------------

def window_mask(T, size):
    i = torch.arange(T)
    dist = i[:, None] - i[None, :]
    seen = dist >= 0
    return seen if size is None else seen & (dist < size)


def masked_attention(q, k, v, scale, seen):
    """q, k [T, H, d], v [T, H, e] -> [T, H, e]."""
    s = (q.transpose(0, 1) @ k.permute(1, 2, 0)) * scale
    p = torch.softmax(s.masked_fill(~seen, float("-inf")), -1)
    return (p @ v.transpose(0, 1)).transpose(0, 1)


def lambda_of(W, p, diff):
    return torch.exp((W[p + "lq1"] * W[p + "lk1"]).sum()) - \
        torch.exp((W[p + "lq2"] * W[p + "lk2"]).sum()) + diff


def diff_attention(h, W, p, m, eps):
    T, H, G, d, e = (h.shape[0], m["heads"], m["kv_heads"], m["dim"],
                     m["vdim"])
    of = [i // (H // G) for i in range(H)]

    def part(name):
        return causal_conv(h @ W[p + name].T + W[p + name + ".b"],
                           W[p + name + ".conv"])

    q = part("q").reshape(T, H, 2, d)
    k = part("k").reshape(T, G, 2, d)[:, of]
    v = part("v").reshape(T, G, e)[:, of]
    seen = window_mask(T, (m.get("mask") or {}).get("size"))
    a1, a2 = (masked_attention(q[:, :, i], k[:, :, i], v, m["scale"], seen)
              for i in (0, 1))
    o = rms(a1 - lambda_of(W, p, m["diff"]) * a2, eps) * (1 - m["diff"])
    return o.reshape(T, H * e) @ W[p + "o"].T


# --- latent attention without positions ----------------------------------------

def latent_attention(h, W, p, m, eps):
    T, H, d, e = h.shape[0], m["heads"], m["dim"], m["vdim"]
    cq = rms(h @ W[p + "dq"].T, eps) * W[p + "dq.norm"]
    c = rms(h @ W[p + "dkv"].T, eps) * W[p + "dkv.norm"]
    q = (cq @ W[p + "uq"].T).reshape(T, H, d)
    k = (c @ W[p + "uk"].T).reshape(T, H, d)
    v = (c @ W[p + "uv"].T).reshape(T, H, e)
    o = masked_attention(q, k, v, m["scale"], window_mask(T, None))
    o = o * torch.sigmoid(h @ W[p + "g"].T)[:, :, None]
    return o.reshape(T, H * e) @ W[p + "o"].T


# --- feed-forward ---------------------------------------------------------------

def poly_norm(z, act, eps):
    a, b, c, e = act
    return a * rms(z, eps) + b * rms(z ** 2, eps) + c * rms(z ** 3, eps) + e


def feed_forward(h, W, p, eps):
    return poly_norm(h @ W[p + "up"].T, W[p + "act"], eps) @ W[p + "down"].T


# --- the model --------------------------------------------------------------------

MIXERS = {"general_delta": general_delta, "attention": diff_attention,
          "latent_attention": latent_attention}


def layer(x, W, p, lay, eps):
    y = MIXERS[lay["type"]](
        canon(centered_norm(x, W[p + "norm1"], eps), W[p + "canon1"]),
        W, p + "mix.", lay["mixer"], eps)
    if lay.get("mlp") is not None:
        y = y + feed_forward(
            canon(centered_norm(x, W[p + "norm2"], eps), W[p + "canon2"]),
            W, p + "mlp.", eps)
    return x + y


def enter_pass(x, x0, W, t):
    return torch.cat([x, x0], -1) @ W["loop.in"].T + W["loop.step"][t]


def softcap(z, cap):
    return z if cap is None else cap * torch.tanh(z / cap)


def forward(cfg, W, tokens, dtype=torch.float64, layers_out=None):
    """Logits [T, vocab] of one sequence; `layers_out` collects the residual
    after every layer run."""
    W = {k: (v.to(dtype) if v.is_floating_point() else v)
         for k, v in W.items()}
    eps, loop, n = cfg["norm"]["eps"], cfg.get("loop"), len(cfg["layers"])
    x = x0 = W["embed"][torch.as_tensor(tokens, dtype=torch.long)]

    def run(x, i):
        x = layer(x, W, f"l{i}.", cfg["layers"][i], eps)
        if layers_out is not None:
            layers_out.append(x)
        return x

    start, stop, times = ((loop["start"], loop["stop"], loop["times"])
                          if loop else (n, n, 0))
    for i in range(start):
        x = run(x, i)
    for t in range(times):
        x = enter_pass(x, x0, W, t)
        for i in range(start, stop):
            x = run(x, i)
    for i in range(stop, n):
        x = run(x, i)
    logits = centered_norm(x, W["final.norm"], eps) @ W["head"].T
    return softcap(logits, cfg.get("logit_softcap"))


# --- small models for the tests ------------------------------------------------

def dense(ff):
    return {"kind": "dense", "ff": ff}


def delta(heads, dim, mlp=None):
    return {"type": "general_delta", "mlp": mlp,
            "mixer": {"heads": heads, "dim": dim}}


def diff(heads, kv_heads, dim, vdim, size, taps=3, diff=0.4, scale=None,
         mlp=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim,
         "conv": taps, "diff": diff,
         "scale": dim ** -0.5 if scale is None else scale}
    if size is not None:
        m["mask"] = {"size": size}
    return {"type": "attention", "mlp": mlp, "mixer": m}


def latent(heads, dim, vdim, q_rank, kv_rank, scale=None, mlp=None):
    return {"type": "latent_attention", "mlp": mlp,
            "mixer": {"heads": heads, "dim": dim, "vdim": vdim,
                      "q_rank": q_rank, "kv_rank": kv_rank,
                      "scale": dim ** -0.5 if scale is None else scale}}


def make_config(layers, width, vocab, loop=None, taps=4, cap=20.0, eps=1e-5):
    """`loop`: (start, stop, times)."""
    out = {"architecture": "Dopilorn", "canon": {"taps": taps},
           "layers": layers, "logit_softcap": cap, "norm": {"eps": eps},
           "vocab": vocab, "width": width}
    if loop is not None:
        out["loop"] = dict(zip(("start", "stop", "times"), loop))
    return out


def make_weights(cfg, seed=0, gain=1.0, rank=6, dtype=torch.bfloat16):
    """`rank`: inner size of the decay projection."""
    g = torch.Generator().manual_seed(seed)

    def lin(o, i, k=1.0):
        return (torch.randn(o, i, generator=g) * gain * k / i ** 0.5
                ).to(dtype)

    def vec(n, mean=1.0, dev=0.3):
        return (mean + dev * torch.randn(n, generator=g)).to(dtype)

    D, V, loop = cfg["width"], cfg["vocab"], cfg.get("loop")
    W = {"embed": lin(V, D, D ** 0.5), "head": lin(V, D, 3),
         "final.norm": vec(D, 0.1)}
    if loop is not None:
        W["loop.in"] = lin(D, 2 * D)
        W["loop.step"] = vec((loop["times"], D), 0.0)
    for i, lay in enumerate(cfg["layers"]):
        m, L, p = lay["mixer"], f"l{i}.", f"l{i}.mix."
        for n in (1, 2) if lay.get("mlp") is not None else (1,):
            W[f"{L}norm{n}"] = vec(D, 0.1)
            W[f"{L}canon{n}"] = vec((D, cfg["canon"]["taps"]), 0.1)
        H, d = m["heads"], m["dim"]
        if lay["type"] == "general_delta":
            for name, k in (("r", 1), ("k", 1), ("v", 1), ("g", 2), ("a", 2)):
                W[p + name] = lin(H * d, D, k)
            W[p + "a.b"], W[p + "w0"] = vec(H * d, 0.5), vec(H * d, -1.5, 1)
            W[p + "w1"], W[p + "w2"] = lin(rank, D), lin(H * d, rank, 2)
            W[p + "norm"], W[p + "o"] = vec(H * d), lin(D, H * d)
        elif lay["type"] == "attention":
            G, e = m["kv_heads"], m["vdim"]
            for name, n in (("q", 2 * H * d), ("k", 2 * G * d), ("v", G * e)):
                W[p + name], W[p + name + ".b"] = lin(n, D, 1.5), vec(n, 0.0)
                W[p + name + ".conv"] = vec((n, m["conv"]), 0.3, 0.5)
            for name in ("lq1", "lk1", "lq2", "lk2"):
                W[p + name] = vec(d, 0.0, d ** -0.25)
            W[p + "o"] = lin(D, H * e)
        else:
            e, rq, r = m["vdim"], m["q_rank"], m["kv_rank"]
            W[p + "dq"], W[p + "dq.norm"] = lin(rq, D), vec(rq)
            W[p + "dkv"], W[p + "dkv.norm"] = lin(r, D), vec(r)
            W[p + "uq"], W[p + "uk"] = lin(H * d, rq, 1.5), lin(H * d, r, 1.5)
            W[p + "uv"], W[p + "g"] = lin(H * e, r, 2), lin(H, D, 2)
            W[p + "o"] = lin(D, H * e)
        if lay.get("mlp") is not None:
            ff = lay["mlp"]["ff"]
            W[f"{L}mlp.up"], W[f"{L}mlp.down"] = lin(ff, D), lin(D, ff)
            W[f"{L}mlp.act"] = vec(4, 0.3, 0.3)
    return W
