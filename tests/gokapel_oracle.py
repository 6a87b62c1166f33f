"""Plain, slow reference of the Gokapel design, written from its equations.

One function per mechanism, whole sequences only, no cache, no batching,
nothing shared with the product path. Weights come as a dict of tensors
under the design's own names ('l0.mix.q', ...), the configuration as the
parsed config.json. Everything runs in the dtype the caller gives (float64
by default), so it serves as the numerics oracle of the tests.
"""
from __future__ import annotations

import torch


def silu(x):
    return x * torch.sigmoid(x)


def rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def dynamic_tanh(x, w, b, alpha):
    return torch.tanh(alpha * x) * w + b


# --- gated delta rule with a decay per channel ------------------------------

def short_conv(x, w):
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


def unit(x):
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


def delta_recurrence(q, k, v, beta, g):
    """q, k, g [T, H, d], v [T, H, e], beta [T, H] -> [T, H, e]."""
    T, H, d = q.shape
    S = torch.zeros(H, d, v.shape[2], dtype=q.dtype)
    out = torch.zeros_like(v)
    for t in range(T):
        S = g[t][:, :, None] * S
        u = beta[t][:, None] * (v[t] - (S * k[t][:, :, None]).sum(1))
        S = S + k[t][:, :, None] * u[:, None, :]
        out[t] = (S * q[t][:, :, None]).sum(1)
    return out


def log_decay(h, W, p, H, d):
    a = h @ W[p + "a1"].T @ W[p + "a2"].T + W[p + "dt_bias"]
    soft = torch.logaddexp(a, torch.zeros_like(a))
    return -torch.exp(W[p + "A_log"])[:, None] * soft.reshape(-1, H, d)


def channel_delta(h, W, p, m, eps):
    T, H, G, d, e = (h.shape[0], m["heads"], m["kv_heads"], m["dim"],
                     m["vdim"])
    of = [i // (H // G) for i in range(H)]

    def part(name):
        return silu(short_conv(h @ W[p + name].T, W[p + name + ".conv"]))

    q = unit(part("q").reshape(T, G, d))[:, of] * d ** -0.5
    k = unit(part("k").reshape(T, G, d))[:, of]
    v = part("v").reshape(T, H, e)
    beta = torch.sigmoid(h @ W[p + "b"].T)
    g = torch.exp(log_decay(h, W, p, H, d))
    o = rms(delta_recurrence(q, k, v, beta, g), eps) * W[p + "norm"]
    gate = torch.sigmoid(h @ W[p + "g1"].T @ W[p + "g2"].T)
    return (o.reshape(T, H * e) * gate) @ W[p + "o"].T


# --- chunked attention with a sink ------------------------------------------

def rotate_pairs(x, rot):
    """x [T, H, d]: dimension 2i turns with 2i + 1, those from `dims` on
    pass."""
    out = x.clone()
    pos = torch.arange(x.shape[0], dtype=x.dtype)[:, None]
    for i in range(rot["dims"] // 2):
        ang = pos * float(rot["base"]) ** (-2.0 * i / rot["dims"])
        u, v = x[..., 2 * i], x[..., 2 * i + 1]
        out[..., 2 * i] = u * torch.cos(ang) - v * torch.sin(ang)
        out[..., 2 * i + 1] = v * torch.cos(ang) + u * torch.sin(ang)
    return out


def chunk_mask(T, size):
    i = torch.arange(T)
    seen = i[None, :] <= i[:, None]
    if size is not None:
        seen = seen & (i[None, :] // size == i[:, None] // size)
    return seen


def sink_softmax(s, sink):
    """s [H, T, T] scores (-inf where hidden), sink [H]: one more entry of
    the denominator."""
    top = torch.maximum(s.max(-1).values, sink[:, None])
    p = torch.exp(s - top[..., None])
    return p / (p.sum(-1) + torch.exp(sink[:, None] - top))[..., None]


def chunked_attention(h, W, p, m, eps):
    T, H, G, d, e = (h.shape[0], m["heads"], m["kv_heads"], m["dim"],
                     m["vdim"])
    of = [i // (H // G) for i in range(H)]
    q = rms((h @ W[p + "q"].T).reshape(T, H, d), eps) * W[p + "q.norm"]
    k = rms((h @ W[p + "k"].T).reshape(T, G, d), eps) * W[p + "k.norm"]
    v = (h @ W[p + "v"].T).reshape(T, G, e)[:, of]
    q, k = rotate_pairs(q, m["rot"]), rotate_pairs(k, m["rot"])[:, of]
    s = (q.transpose(0, 1) @ k.permute(1, 2, 0)) * m["scale"]
    s = s.masked_fill(~chunk_mask(T, (m.get("mask") or {}).get("size")),
                      float("-inf"))
    a = sink_softmax(s, W[p + "sink"])
    o = (a @ v.transpose(0, 1)).transpose(0, 1)
    return o.reshape(T, H * e) @ W[p + "o"].T


# --- minGRU ------------------------------------------------------------------

def gated_recurrence(z, cand):
    S, out = torch.zeros_like(z[0]), torch.zeros_like(z)
    for t in range(z.shape[0]):
        S = (1 - z[t]) * S + z[t] * cand[t]
        out[t] = S
    return out


def min_gru(h, W, p):
    z = torch.sigmoid(h @ W[p + "z"].T + W[p + "z.b"])
    u = h @ W[p + "x"].T + W[p + "x.b"]
    cand = torch.where(u >= 0, u + 0.5, torch.sigmoid(u))
    return (gated_recurrence(z, cand) * silu(h @ W[p + "g"].T)) @ \
        W[p + "o"].T


def parallel(h, W, p, m, eps):
    return m["left_scale"] * chunked_attention(h, W, p + "left.", m["left"],
                                               eps) + \
        m["right_scale"] * min_gru(h, W, p + "right.")


# --- feed-forward ------------------------------------------------------------

def squared_relu(h, W, p):
    return torch.relu(h @ W[p + "up"].T) ** 2 @ W[p + "down"].T


def choose(z, correction, r):
    """z [experts] logits of one token -> (chosen experts, their weights)."""
    E = r["experts"]
    s = torch.softmax(z, -1)
    choice = (s + correction).tolist()
    allowed = list(range(E))
    if r.get("groups"):
        n = E // r["groups"]["count"]
        best = [max(choice[i:i + n]) for i in range(0, E, n)]
        kept = sorted(range(len(best)), key=lambda i: -best[i])
        kept = kept[:r["groups"]["keep"]]
        allowed = [e for e in allowed if e // n in kept]
    picked = sorted(allowed, key=lambda e: -choice[e])[:r["top"]]
    return picked, [s[e] for e in picked]


def mixture(h, W, p, m):
    out = torch.zeros_like(h)
    z = h @ W[p + "router"].T
    for t in range(h.shape[0]):
        for e, w in zip(*choose(z[t], W[p + "correction"], m["router"])):
            out[t] = out[t] + w * squared_relu(h[t], W, f"{p}e{e}.")
    if m.get("shared"):
        out = out + squared_relu(h, W, p + "shared.")
    return out


# --- streams -----------------------------------------------------------------

def spread(X, y, mix, out, mult):
    """X [T, s, D]: every stream from all the old ones and the sublayer's
    result; mix is indexed [from, to]."""
    s = X.shape[1]
    new = torch.zeros_like(X)
    for t in range(s):
        for f in range(s):
            new[:, t] = new[:, t] + mix[f, t] * X[:, f]
        new[:, t] = new[:, t] + mult * out[t] * y
    return new


def forward(cfg, W, tokens, dtype=torch.float64, layers_out=None):
    """Logits [T, vocab] of one sequence; `layers_out` collects the sum of
    the streams after every layer."""
    W = {k: (v.to(dtype) if v.is_floating_point() else v)
         for k, v in W.items()}
    eps, mult = cfg["norm"]["eps"], cfg["residual_mult"]

    def norm(x, n):
        return dynamic_tanh(x, W[n], W[n + ".b"], W[n + ".alpha"])

    x = W["embed"][torch.as_tensor(tokens, dtype=torch.long)] * \
        cfg["embedding"]["scale"]
    X = x[:, None].repeat(1, cfg["streams"], 1)
    for i, lay in enumerate(cfg["layers"]):
        p = f"l{lay.get('weights_of', i)}."

        def sublayer(X, n, f):
            hc = f"{p}hc{n}."
            u = (X * W[hc + "in"][None, :, None]).sum(1)
            h = norm(u, f"{p}norm{n}")
            gate = torch.sigmoid(h @ W[f"{p}rg{n}"].T + W[f"{p}rg{n}.b"])
            y = f(h) * W[f"{p}ls{n}"] * gate
            return spread(X, y, W[hc + "mix"], W[hc + "out"], mult)

        mixer = {"channel_delta": channel_delta,
                 "parallel": parallel}[lay["type"]]
        X = sublayer(X, 1, lambda h: mixer(h, W, p + "mix.", lay["mixer"],
                                           eps))
        mlp = lay.get("mlp")
        if mlp is not None:
            X = sublayer(X, 2, (lambda h: squared_relu(h, W, p + "mlp."))
                         if mlp["kind"] == "dense" else
                         (lambda h: mixture(h, W, p + "mlp.", mlp)))
        if layers_out is not None:
            layers_out.append(X.sum(1))
    return norm(X.sum(1), "final.norm") @ W["embed"].T


# --- small models for the tests ---------------------------------------------

def delta(heads, kv_heads, dim, vdim, taps=4, mlp=None, weights_of=None):
    lay = {"type": "channel_delta", "mlp": mlp,
           "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim,
                     "vdim": vdim, "conv": taps}}
    if weights_of is not None:
        lay["weights_of"] = weights_of
    return lay


def twin(heads, kv_heads, dim, vdim, size, rot, width, base=10000.0,
         scale=None, scales=(0.7, 0.4), mlp=None, weights_of=None):
    left = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim,
            "scale": dim ** -0.5 if scale is None else scale,
            "rot": {"base": base, "dims": rot}}
    if size is not None:
        left["mask"] = {"size": size}
    lay = {"type": "parallel", "mlp": mlp,
           "mixer": {"left": left, "left_scale": scales[0],
                     "right": {"width": width}, "right_scale": scales[1]}}
    if weights_of is not None:
        lay["weights_of"] = weights_of
    return lay


def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(ff, experts, top, groups=None, shared=None):
    """`groups`: (count, keep) or None."""
    router = {"experts": experts, "top": top}
    if groups is not None:
        router["groups"] = {"count": groups[0], "keep": groups[1]}
    out = {"kind": "moe", "expert": {"ff": ff}, "router": router}
    if shared is not None:
        out["shared"] = {"ff": shared}
    return out


def make_config(layers, width, vocab, streams=3, mult=0.8, embed_scale=3.0,
                eps=1e-5):
    return {"architecture": "Gokapel", "embedding": {"scale": embed_scale},
            "layers": layers, "norm": {"eps": eps}, "residual_mult": mult,
            "streams": streams, "vocab": vocab, "width": width}


def make_weights(cfg, seed=0, gain=1.0, ranks=(6, 10), dtype=torch.bfloat16):
    """`ranks`: inner sizes of the decay and gate projections."""
    g = torch.Generator().manual_seed(seed)

    def lin(o, i, k=1.0):
        return (torch.randn(o, i, generator=g) * gain * k / i ** 0.5
                ).to(dtype)

    def vec(n, mean=1.0, dev=0.3):
        return (mean + dev * torch.randn(n, generator=g)).to(dtype)

    D, V, s = cfg["width"], cfg["vocab"], cfg["streams"]
    W = {"embed": lin(V, D, D ** 0.5 / cfg["embedding"]["scale"])}

    def norm(name):
        W[name], W[name + ".b"] = vec(D), vec(D, 0.0)
        W[name + ".alpha"] = vec(1, 0.7, 0.1)[0]

    norm("final.norm")
    for i, lay in enumerate(cfg["layers"]):
        if "weights_of" in lay:
            continue
        m, L, mlp = lay["mixer"], f"l{i}.", lay.get("mlp")
        for n in (1, 2) if mlp is not None else (1,):
            norm(f"{L}norm{n}")
            W[f"{L}ls{n}"] = vec(D)
            W[f"{L}rg{n}"], W[f"{L}rg{n}.b"] = lin(D, D), vec(D, 0.5)
            W[f"{L}hc{n}.in"] = vec(s, 1 / s, 0.3)
            W[f"{L}hc{n}.out"] = vec(s)
            W[f"{L}hc{n}.mix"] = (0.8 * torch.eye(s) + 0.15 * torch.randn(
                s, s, generator=g)).to(dtype)
        p = L + "mix."
        if lay["type"] == "channel_delta":
            H, G, d, e = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
            for name, n in (("q", G * d), ("k", G * d), ("v", H * e)):
                W[p + name] = lin(n, D, 2)
                W[p + name + ".conv"] = vec((n, m["conv"]), 0.2, 0.5)
            W[p + "b"] = lin(H, D)
            W[p + "A_log"] = vec(H, -0.5, 1.0)
            W[p + "dt_bias"] = vec(H * d, -2.0, 1.0)
            W[p + "norm"] = vec(e)
            W[p + "a1"], W[p + "a2"] = lin(ranks[0], D), lin(H * d, ranks[0])
            W[p + "g1"], W[p + "g2"] = lin(ranks[1], D), lin(H * e, ranks[1])
            W[p + "o"] = lin(D, H * e, 2)
        else:
            a, R, q = m["left"], m["right"]["width"], p + "left."
            H, G, d, e = a["heads"], a["kv_heads"], a["dim"], a["vdim"]
            W[q + "q"], W[q + "k"] = lin(H * d, D), lin(G * d, D)
            W[q + "v"], W[q + "o"] = lin(G * e, D, 2), lin(D, H * e, 2)
            W[q + "q.norm"], W[q + "k.norm"] = vec(d, 1.5), vec(d, 1.5)
            W[q + "sink"] = vec(H, 0.0, 1.5)
            q = p + "right."
            W[q + "z"], W[q + "z.b"] = lin(R, D), vec(R, -1.0)
            W[q + "x"], W[q + "x.b"] = lin(R, D, 2), vec(R, 0.0)
            W[q + "g"], W[q + "o"] = lin(R, D, 2), lin(D, R, 2)
        if mlp is None:
            continue
        p = L + "mlp."

        def ffn(q, F):
            W[q + "up"], W[q + "down"] = lin(F, D, 1.5), lin(D, F)

        if mlp["kind"] == "dense":
            ffn(p, mlp["ff"])
            continue
        E = mlp["router"]["experts"]
        W[p + "router"], W[p + "correction"] = lin(E, D, 3), vec(E, 0, 0.05)
        for x in range(E):
            ffn(f"{p}e{x}.", mlp["expert"]["ff"])
        if mlp.get("shared"):
            ffn(p + "shared.", mlp["shared"]["ff"])
    return W
