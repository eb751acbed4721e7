"""Plain, slow implementation of the Pifazen decoder, one function per mechanism.

Everything runs over whole sequences without a cache, in the dtype of the weights it is given
(the tests use float64).  It shares no code with the package: it is what the product path is
compared against.

Notation: W width, H / G value and query-key heads, d / v key and value sizes of a head.
"""
from __future__ import annotations

import math

import torch


def sigmoid(z):
    return 1 / (1 + torch.exp(-z))


def softplus(z):
    return torch.clamp(z, min=0) + torch.log1p(torch.exp(-z.abs()))


def unit_rms(x, eps):
    """x over its root mean square along the last axis, eps inside the root."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def layer_norm(x, w, eps):
    """The layers' norm: its weight is stored as the distance from one."""
    return unit_rms(x, eps) * (1 + w)


def _under(t, prefix):
    return {k[len(prefix):]: v for k, v in t.items() if k.startswith(prefix)}


# ------------------------------------------------------------------ rotation
def frequencies(rot):
    """(angle a position of every pair, factor on cosines and sines)."""
    n, base = rot["dims"], rot["base"]
    f = [base ** (-2 * i / n) for i in range(n // 2)]
    sc = rot.get("scaling")
    if not sc:
        return f, 1.0

    def dim(turns):
        return n * math.log(sc["original"] / (2 * math.pi * turns)) / (2 * math.log(base))

    lo, hi = max(math.floor(dim(sc["fast"])), 0), min(math.ceil(dim(sc["slow"])), n - 1)
    out = []
    for i, fi in enumerate(f):
        ramp = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(fi / sc["factor"] * ramp + fi * (1 - ramp))
    return out, 0.1 * math.log(sc["factor"]) + 1


def rotate(x, rot):
    """x [T, heads, r]: neighbours (2i, 2i + 1) turned by position."""
    f, m = frequencies(rot)
    a = torch.arange(x.shape[0], dtype=torch.float64)[:, None] * torch.tensor(f, dtype=torch.float64)
    c, s = (m * torch.cos(a)).to(x.dtype)[:, None], (m * torch.sin(a)).to(x.dtype)[:, None]
    u, v = x[..., 0::2], x[..., 1::2]
    return torch.stack([u * c - v * s, v * c + u * s], -1).reshape(x.shape)


# ------------------------------------------------------------------ latent attention
def attend(qu, qr, ku, kr, v, scale):
    """Causal softmax attention, a score from the heads' own keys and the shared rotated key:
    qu [T, H, d], qr [T, H, r], ku [T, H, d], kr [T, r], v [T, H, vd]."""
    T, H = qu.shape[:2]
    out = torch.zeros(T, H, v.shape[-1], dtype=qu.dtype)
    later = torch.ones(T, T, dtype=torch.bool).triu(1)
    for h in range(H):
        s = (qu[:, h] @ ku[:, h].T + qr[:, h] @ kr.T) * scale
        s = s.masked_fill(later, -math.inf)
        p = torch.exp(s - s.max(-1, keepdim=True).values)
        out[:, h] = (p @ v[:, h]) / p.sum(-1, keepdim=True)
    return out


def latent_attention(h, m, t, eps):
    """``t`` its tensors: queries from h, or (with "dq") from a normed latent of h; the gate one
    number an output element, or one a head -- as many rows as its tensor has."""
    T, H, d, r, R = h.shape[0], m["heads"], m["dim"], m["rot_dim"], m["kv_rank"]
    q = (unit_rms(h @ t["dq"].T, eps) * t["dq.norm"]) @ t["uq"].T if "dq" in t else h @ t["q"].T
    q = q.view(T, H, d + r)
    z = h @ t["dkv"].T
    c = unit_rms(z[:, :R], eps) * t["dkv.norm"]
    qr, kr = rotate(q[..., d:], m["rot"]), rotate(z[:, None, R:], m["rot"])[:, 0]
    o = attend(q[..., :d], qr, (c @ t["uk"].T).view(T, H, d), kr, (c @ t["uv"].T).view(T, H, m["vdim"]), m["scale"])
    return (o * sigmoid(h @ t["g"].T).view(T, H, -1)).reshape(T, -1) @ t["o"].T


# ------------------------------------------------------------------ channel delta rule
def delta_recurrence(q, k, v, g, beta):
    """S <- diag(g) S; u = beta (v - S^T k); S <- S + k u^T; o = S^T q; q, k, g [T, H, d], beta [T, H]."""
    T, H, d = q.shape
    S = torch.zeros(H, d, v.shape[-1], dtype=q.dtype)
    out = torch.zeros(T, H, v.shape[-1], dtype=q.dtype)
    for t in range(T):
        S = g[t][..., None] * S
        u = beta[t][:, None] * (v[t] - torch.einsum("hdv,hd->hv", S, k[t]))
        S = S + k[t][..., None] * u[:, None]
        out[t] = torch.einsum("hdv,hd->hv", S, q[t])
    return out


def short_conv(x, w):
    """silu of the causal convolution per channel; the last tap weighs the current token."""
    taps = w.shape[1]
    y = torch.zeros_like(x)
    for back in range(taps):
        if back < x.shape[0]:
            y[back:] += x[:x.shape[0] - back] * w[:, taps - 1 - back]
    return y * sigmoid(y)


def unit(x):
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


def channel_decay(h, t, H, d):
    z = (h @ t["a1"].T) @ t["a2"].T + t["dt_bias"]
    return torch.exp(-torch.exp(t["A_log"])[None, :, None] * softplus(z).view(h.shape[0], H, d))


def channel_delta(h, m, t, eps):
    T, H, G, d = h.shape[0], m["heads"], m["kv_heads"], m["dim"]
    q, k, v = (short_conv(h @ t[n].T, t[n + ".conv"]) for n in "qkv")
    q, k = (unit(x.view(T, G, d)).repeat_interleave(H // G, 1) for x in (q, k))
    o = delta_recurrence(q * d ** -0.5, k, v.view(T, H, m["vdim"]), channel_decay(h, t, H, d), sigmoid(h @ t["b"].T))
    o = (unit_rms(o, eps) * t["norm"]).reshape(T, -1)
    return (o * sigmoid((h @ t["g1"].T) @ t["g2"].T)) @ t["o"].T


MIXERS = {"channel_delta": channel_delta, "latent_attention": latent_attention, "latent_attention_2": latent_attention}


# ------------------------------------------------------------------ feed-forwards
def poly_norm(z, act, eps):
    a, b, c, e = act
    return a * unit_rms(z, eps) + b * unit_rms(z ** 2, eps) + c * unit_rms(z ** 3, eps) + e


def dense(h, t, eps):
    return poly_norm(h @ t["up"].T + t["up.b"], t["act"], eps) @ t["down"].T + t["down.b"]


def expert(h, t, limit):
    g = torch.clamp(h @ t["gate"].T, max=limit)
    u = torch.clamp(h @ t["up"].T, -limit, limit)
    return (g * sigmoid(1.702 * g) * (u + 1)) @ t["down"].T


def route(h, r, t):
    """(chosen [T, top], their weights)."""
    z = h @ t["router"].T
    s = torch.exp(z - z.max(-1, keepdim=True).values)
    s = s / s.sum(-1, keepdim=True)
    choice = s + t["correction"]
    n, gr = choice.shape[1], r["groups"]
    parts = choice.view(-1, gr["count"], n // gr["count"])
    keep = torch.topk(parts.max(-1).values, gr["keep"], -1).indices
    alive = torch.zeros(parts.shape[:2], dtype=torch.bool).scatter(1, keep, True)
    choice = parts.masked_fill(~alive[..., None], -math.inf).reshape(-1, n)
    best = torch.topk(choice, r["top"], -1).indices
    w = s.gather(1, best)
    return best, w / (w.sum(-1, keepdim=True) + 1e-20) * r["scale"]


def experts(h, m, t):
    r = m["router"]
    best, w = route(h, r, t)
    y = torch.zeros_like(h)
    for e in range(r["experts"] + r["identity"]):
        share = (w * (best == e)).sum(-1, keepdim=True)
        rows = share[:, 0] != 0
        if rows.any():
            out = expert(h[rows], _under(t, f"e{e}."), m["expert"]["limit"]) if e < r["experts"] else h[rows]
            y[rows] += share[rows] * out
    return y


# ------------------------------------------------------------------ the model
def forward(cfg, weights, tokens, dtype=torch.float64, residuals=None):
    """logits [T, vocab]; ``residuals``: a list that receives the stream after every layer."""
    w = {k: v.to(dtype) for k, v in weights.items()}
    eps = cfg["norm"]["eps"]
    x = w["embed"][torch.as_tensor(tokens, dtype=torch.long)]
    for i, L in enumerate(cfg["layers"]):
        t = _under(w, f"l{L.get('weights_of', i)}.")
        x = x + t["ls1"] * MIXERS[L["type"]](layer_norm(x, t["norm1"], eps), L["mixer"], _under(t, "mix."), eps)
        f = L.get("mlp")
        if f:
            h, ft = layer_norm(x, t["norm2"], eps), _under(t, "mlp.")
            x = x + t["ls2"] * (dense(h, ft, eps) if f["kind"] == "dense" else experts(h, f, ft))
        if residuals is not None:
            residuals.append(x)
    return layer_norm(x, w["final.norm"], eps) @ w["embed"].T


def random_weights(cfg, seed=0, rank=(5, 7), dtype=torch.float32):
    """Random weights of the tensors ``cfg`` names, sized so that every mechanism matters; ``rank``:
    inner sizes of the decay's and the gate's projections."""
    g = torch.Generator().manual_seed(seed)

    def nrm(*shape, s=1.0):
        return torch.randn(*shape, generator=g) * s

    def lin(n, k, s=1.0):
        return nrm(n, k, s=s * k ** -0.5)

    W, V = cfg["width"], cfg["vocab"]
    w = {"embed": nrm(V, W), "final.norm": nrm(W, s=0.2)}
    for i, L in enumerate(cfg["layers"]):
        if "weights_of" in L:
            continue
        p, m, f = f"l{i}.", L["mixer"], L.get("mlp")
        x = p + "mix."
        w.update({p + "norm1": nrm(W, s=0.2), p + "ls1": 1 + nrm(W, s=0.3)})
        H, vd = m["heads"], m["vdim"]
        w[x + "o"] = lin(W, H * vd, 1.5)
        if L["type"] == "channel_delta":
            G, d = m["kv_heads"], m["dim"]
            for n, rows in (("q", G * d), ("k", G * d), ("v", H * vd)):
                w.update({x + n: lin(rows, W), x + n + ".conv": nrm(rows, m["conv"], s=0.6)})
            w.update({x + "b": lin(H, W), x + "A_log": nrm(H, s=0.5) - 1, x + "dt_bias": nrm(H * d) - 2, x + "norm": 1 + nrm(vd, s=0.2),
                      x + "a1": lin(rank[0], W), x + "a2": lin(H * d, rank[0], 1.5), x + "g1": lin(rank[1], W),
                      x + "g2": lin(H * vd, rank[1], 1.5)})
        else:
            d, r, R = m["dim"], m["rot_dim"], m["kv_rank"]
            rows = H * (d + r)
            if L["type"] == "latent_attention":
                Q = m["q_rank"]
                w.update({x + "dq": lin(Q, W), x + "dq.norm": 1.5 + nrm(Q, s=0.3), x + "uq": lin(rows, Q, 1.3), x + "g": lin(H * vd, W)})
            else:
                w.update({x + "q": lin(rows, W, 1.5), x + "g": lin(H, W)})
            w.update({x + "dkv": lin(R + r, W, 1.5), x + "dkv.norm": 1 + nrm(R, s=0.2), x + "uk": lin(H * d, R, 1.5), x + "uv": lin(H * vd, R)})
        if f is None:
            continue
        x = p + "mlp."
        w.update({p + "norm2": nrm(W, s=0.2), p + "ls2": 1 + nrm(W, s=0.3)})
        if f["kind"] == "dense":
            F = f["ff"]
            w.update({x + "up": lin(F, W), x + "up.b": nrm(F, s=0.3), x + "down": lin(W, F, 1.5), x + "down.b": nrm(W, s=0.3),
                      x + "act": torch.tensor([0.7, 0.5, 0.4, 0.1]) + nrm(4, s=0.05)})
            continue
        r, F = f["router"], f["expert"]["ff"]
        n = r["experts"] + r["identity"]
        w.update({x + "router": lin(n, W, 2.0), x + "correction": nrm(n, s=0.2)})
        for e in range(r["experts"]):
            w.update({f"{x}e{e}.gate": lin(F, W, 1.5), f"{x}e{e}.up": lin(F, W, 1.5), f"{x}e{e}.down": lin(W, F, 1.5)})
    return {k: v.to(torch.bfloat16).to(dtype) for k, v in w.items()}
