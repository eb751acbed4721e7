"""Plain, slow implementation of the Gezozen decoder, one function per mechanism.

Everything runs over whole sequences without a cache, in the dtype of the weights it is given
(the tests use float64).  It shares no code with the package: it is what the product path is
compared against.

Notation: W width, H / G query and key-value heads, d / v key and value sizes of a head.
"""
from __future__ import annotations

import math

import torch


def sigmoid(z):
    return 1 / (1 + torch.exp(-z))


def silu(z):
    return z * sigmoid(z)


def softplus(z):
    return torch.clamp(z, min=0) + torch.log1p(torch.exp(-z.abs()))


def rms(x, eps):
    """x scaled to unit root mean square over its last axis; eps is added inside the root."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def group_norm(x, w, groups, eps):
    """RMS norm of each of ``groups`` equal consecutive parts, then the weight over the whole."""
    return rms(x.view(*x.shape[:-1], groups, -1), eps).reshape(x.shape) * w


def after_sum(x, y, gate_w, gate_b, alpha, w, groups, eps):
    """The stream after a sublayer: its gated result is added to alpha x, then normed."""
    return group_norm(alpha * x + sigmoid(x @ gate_w.T + gate_b) * y, w, groups, eps)


# ------------------------------------------------------------------ rotation
def frequencies(rot):
    """(angle per position of every pair, factor on cosines and sines)."""
    r, base = rot["dims"], rot["base"]
    f = [base ** (-2 * i / r) for i in range(r // 2)]
    sc = rot.get("scaling")
    if not sc:
        return f, 1.0

    def dim(turns):
        return r * math.log(sc["original"] / (2 * math.pi * turns)) / (2 * math.log(base))

    lo, hi = max(math.floor(dim(sc["fast"])), 0), min(math.ceil(dim(sc["slow"])), r - 1)
    out = []
    for i, fi in enumerate(f):
        ramp = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(fi / sc["factor"] * ramp + fi * (1 - ramp))
    return out, 0.1 * math.log(sc["factor"]) + 1


def rotate(x, rot, start=0):
    """x [T, heads, d]: the first ``dims`` dimensions turned by position, i paired with i + dims/2."""
    r = rot["dims"]
    f, m = frequencies(rot)
    a = torch.arange(start, start + x.shape[0], dtype=torch.float64)[:, None] * torch.tensor(f, dtype=torch.float64)
    c, s = (m * torch.cos(a)).to(x.dtype)[:, None], (m * torch.sin(a)).to(x.dtype)[:, None]
    u, v = x[..., :r // 2], x[..., r // 2:r]
    return torch.cat([u * c - v * s, v * c + u * s, x[..., r:]], -1)


# ------------------------------------------------------------------ attention
def attend(q, k, v, scale, window=0, cap=None):
    """q [T, H, d], k [T, G, d], v [T, G, vd]: causal softmax attention over the last ``window``
    tokens (0: all), scores capped by ``cap``."""
    T, H = q.shape[:2]
    G = k.shape[1]
    out = torch.zeros(T, H, v.shape[-1], dtype=q.dtype)
    for h in range(H):
        g = h // (H // G)
        for i in range(T):
            lo = max(0, i - window + 1) if window else 0
            s = (k[lo:i + 1, g] @ q[i, h]) * scale
            if cap is not None:
                s = cap * torch.tanh(s / cap)
            p = torch.exp(s - s.max())
            out[i, h] = (p @ v[lo:i + 1, g]) / p.sum()
    return out


def attention(h, m, t, eps):
    """The attention side of a parallel mixer; ``t`` its tensors."""
    T, H, G = h.shape[0], m["heads"], m["kv_heads"]

    def proj(name, heads, d):
        y = h @ t[name].T
        return (y + t[name + ".b"] if name + ".b" in t else y).view(T, heads, d)

    q, k, v = proj("q", H, m["dim"]), proj("k", G, m["dim"]), proj("v", G, m["vdim"])
    q, k = rotate(rms(q, eps) * t["q.norm"], m["rot"]), rotate(rms(k, eps) * t["k.norm"], m["rot"])
    o = attend(q, k, v, m["scale"], m.get("mask", {}).get("size", 0), m.get("softcap"))
    return o.reshape(T, -1) @ t["o"].T


# ------------------------------------------------------------------ recurrences
def linear_recurrence(q, k, v, decay):
    """S <- diag(decay) S + k v^T, o = S^T q; q, k, decay [T, H, d], v [T, H, vd]."""
    T, H, d = q.shape
    S = torch.zeros(H, d, v.shape[-1], dtype=q.dtype)
    out = torch.zeros(T, H, v.shape[-1], dtype=q.dtype)
    for t in range(T):
        S = decay[t][..., None] * S + k[t][..., None] * v[t][:, None]
        out[t] = torch.einsum("hdv,hd->hv", S, q[t])
    return out


def delta_recurrence(q, k, v, g, beta):
    """S <- g S; u = beta (v - S^T k); S <- S + k u^T; o = S^T q; q, k [T, H, d], g, beta [T, H]."""
    T, H, d = q.shape
    S = torch.zeros(H, d, v.shape[-1], dtype=q.dtype)
    out = torch.zeros(T, H, v.shape[-1], dtype=q.dtype)
    for t in range(T):
        S = g[t][:, None, None] * S
        u = beta[t][:, None] * (v[t] - torch.einsum("hdv,hd->hv", S, k[t]))
        S = S + k[t][..., None] * u[:, None]
        out[t] = torch.einsum("hdv,hd->hv", S, q[t])
    return out


def read_out(o, h, wg, wo, eps, w=None):
    """Heads normed (times ``w``), gated by silu(W_g h), projected."""
    o = rms(o, eps)
    o = (o if w is None else o * w).reshape(o.shape[0], -1)
    return (o * silu(h @ wg.T)) @ wo.T


def gated_linear(h, m, t, eps):
    T, H, d = h.shape[0], m["heads"], m["dim"]
    q, k = (h @ t["q"].T).view(T, H, d) * d ** -0.5, (h @ t["k"].T).view(T, H, d)
    z = (h @ t["a1"].T) @ t["a2"].T + t["a2.b"]
    decay = (sigmoid(z) ** (1 / m["tau"])).view(T, H, d)
    o = linear_recurrence(q, k, (h @ t["v"].T).view(T, H, m["vdim"]), decay)
    return read_out(o, h, t["g"], t["o"], eps, t["norm"])


def retention(h, m, t, eps):
    T, H, d = h.shape[0], m["heads"], m["dim"]
    q = rotate((h @ t["q"].T).view(T, H, d), m["rot"])
    k = rotate((h @ t["k"].T).view(T, H, d), m["rot"]) * d ** -0.5
    decay = torch.tensor(m["decay"], dtype=h.dtype)[None, :, None].expand(T, H, d)
    o = linear_recurrence(q, k, (h @ t["v"].T).view(T, H, m["vdim"]), decay)
    return read_out(o, h, t["g"], t["o"], eps)


def short_conv(x, w):
    """silu of the causal convolution per channel; the last tap weighs the current token."""
    taps = w.shape[1]
    y = torch.zeros_like(x)
    for back in range(taps):
        if back < x.shape[0]:
            y[back:] += x[:x.shape[0] - back] * w[:, taps - 1 - back]
    return silu(y)


def unit(x):
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


def delta_rule(h, m, t, eps):
    T, H, G, d = h.shape[0], m["heads"], m["kv_heads"], m["dim"]
    q, k, v = (short_conv(h @ t[n].T, t[n + ".conv"]) for n in "qkv")
    q, k = (unit(x.view(T, G, d)).repeat_interleave(H // G, 1) for x in (q, k))
    g = torch.exp(-torch.exp(t["A_log"]) * softplus(h @ t["a"].T + t["dt_bias"]))
    o = delta_recurrence(q * d ** -0.5, k, v.view(T, H, m["vdim"]), g, sigmoid(h @ t["b"].T))
    return read_out(o, h, t["g"], t["o"], eps, t["norm"])


def _under(t, prefix):
    return {k[len(prefix):]: v for k, v in t.items() if k.startswith(prefix)}


def mixer(kind, h, m, t, eps):
    if kind == "delta":
        return delta_rule(h, m, t, eps)
    right = {"parallel": gated_linear, "parallel_2": retention}[kind]
    return (m["left_scale"] * attention(h, m["left"], _under(t, "left."), eps)
            + m["right_scale"] * right(h, m["right"], _under(t, "right."), eps))


# ------------------------------------------------------------------ experts
def expert(h, t):
    return (silu(h @ t["gate"].T) * (h @ t["up"].T)) @ t["down"].T


def experts(h, m, t):
    """Each token's ``top`` experts by sigmoid score, their inputs weighted by it, and the shared
    expert weighted by its own gate."""
    s = sigmoid(h @ t["router"].T)
    best = torch.topk(s, m["router"]["top"], -1).indices
    y = torch.zeros_like(h)
    for e in range(m["router"]["experts"]):
        rows = (best == e).any(-1)
        if rows.any():
            y[rows] += expert(s[rows, e:e + 1] * h[rows], _under(t, f"e{e}."))
    if m.get("shared"):
        y = y + sigmoid(h @ t["shared.sg"].T) * expert(h, _under(t, "shared."))
    return y


# ------------------------------------------------------------------ the model
def forward(cfg, weights, tokens, dtype=torch.float64, residuals=None):
    """logits [T, vocab]; ``residuals``: a list that receives the stream after every layer."""
    w = {k: v.to(dtype) for k, v in weights.items()}
    eps, groups, alpha = cfg["norm"]["eps"], cfg["norm"]["groups"], cfg["postln_alpha"]
    x = w["embed"][torch.as_tensor(tokens, dtype=torch.long)]
    for i, L in enumerate(cfg["layers"]):
        t = _under(w, f"l{i}.")
        y = mixer(L["type"], x, L["mixer"], _under(t, "mix."), eps)
        x = after_sum(x, y, t["rg1"], t["rg1.b"], alpha, t["norm1"], groups, eps)
        if L.get("mlp"):
            y = experts(x, L["mlp"], _under(t, "mlp."))
            x = after_sum(x, y, t["rg2"], t["rg2.b"], alpha, t["norm2"], groups, eps)
        if residuals is not None:
            residuals.append(x)
    return group_norm(x, w["final.norm"], groups, eps) @ w["head"].T


def random_weights(cfg, seed=0, rank=5, dtype=torch.float32):
    """Random weights of the tensors ``cfg`` names, sized so that every mechanism matters."""
    g = torch.Generator().manual_seed(seed)

    def nrm(*shape, s=1.0):
        return torch.randn(*shape, generator=g) * s

    def lin(n, k, s=1.0):
        return nrm(n, k, s=s * k ** -0.5)

    W, V = cfg["width"], cfg["vocab"]
    w = {"embed": nrm(V, W), "head": lin(V, W, 1.5), "final.norm": 1 + nrm(W, s=0.2)}

    def qkv(p, m, s=1.0, kv=None):
        H, G = m["heads"], kv or m["heads"]
        d, vd = m["dim"], m["vdim"]
        hv = G if p.endswith("left.") else H
        w.update({p + "q": lin((H if p.endswith("left.") else G) * d, W, s), p + "k": lin(G * d, W, s), p + "v": lin(hv * vd, W),
                  p + "o": lin(W, H * vd, 1.5)})

    for i, L in enumerate(cfg["layers"]):
        p, m = f"l{i}.", L["mixer"]
        w.update({p + "norm1": 1 + nrm(W, s=0.2), p + "rg1": lin(W, W), p + "rg1.b": nrm(W, s=0.5) + 0.5})
        if L["type"] == "delta":
            x = p + "mix."
            H, G = m["heads"], m["kv_heads"]
            qkv(x, m, kv=G)
            w.update({x + n + ".conv": nrm(c, m["conv"], s=0.6) for n, c in (("q", G * m["dim"]), ("k", G * m["dim"]), ("v", H * m["vdim"]))})
            w.update({x + "b": lin(H, W), x + "a": lin(H, W), x + "A_log": nrm(H, s=0.5) - 1, x + "dt_bias": nrm(H) - 2,
                      x + "norm": 1 + nrm(m["vdim"], s=0.2), x + "g": lin(H * m["vdim"], W)})
        else:
            x, a = p + "mix.left.", m["left"]
            qkv(x, a, 1.0, a["kv_heads"])
            w.update({x + "q.norm": 1.5 + nrm(a["dim"], s=0.3), x + "k.norm": 1.5 + nrm(a["dim"], s=0.3)})
            if L["type"] == "parallel_2":
                w.update({x + n + ".b": nrm(w[x + n].shape[0], s=0.5) for n in "qkv"})
            x, r = p + "mix.right.", m["right"]
            qkv(x, r)
            w[x + "g"] = lin(r["heads"] * r["vdim"], W)
            if L["type"] == "parallel":
                hd = r["heads"] * r["dim"]
                w.update({x + "norm": 1 + nrm(r["vdim"], s=0.2), x + "a1": lin(rank, W), x + "a2": lin(hd, rank, 2.0), x + "a2.b": nrm(hd)})
        if L.get("mlp"):
            f = L["mlp"]
            p2 = p + "mlp."
            w.update({p + "norm2": 1 + nrm(W, s=0.2), p + "rg2": lin(W, W), p + "rg2.b": nrm(W, s=0.5) + 0.5,
                      p2 + "router": lin(f["router"]["experts"], W, 2.0)})
            sizes = {f"e{e}.": f["expert"]["ff"] for e in range(f["router"]["experts"])}
            if f.get("shared"):
                sizes["shared."] = f["shared"]["ff"]
                w[p2 + "shared.sg"] = lin(1, W)
            for n, ff in sizes.items():
                w.update({p2 + n + "gate": lin(ff, W, 1.5), p2 + n + "up": lin(ff, W), p2 + n + "down": lin(W, ff, 1.5)})
    return {k: v.to(torch.bfloat16).to(dtype) for k, v in w.items()}
