"""Plain, slow implementation of the Saritar decoder, one function per mechanism.

Everything runs over whole sequences without a cache, in the dtype of the weights it is
given (the tests use float64 or float32).  It shares no code with the package: it is what
the product path is compared against.

Notation: W width, H / G query / key-value heads, d head size, C channels of the selective
scan, N its states per channel, R the rank of its step projection.
"""
from __future__ import annotations

import math

import torch


def rms(x, eps):
    """x scaled to unit root mean square over its last axis; eps is added inside the root."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def rms_norm(x, w, eps):
    return rms(x, eps) * w


def embed(table, tokens, scale):
    return table[tokens] * scale


def squared_relu(u):
    return torch.clamp(u, min=0) ** 2


def feed_forward(h, up, down):
    return squared_relu(h @ up.T) @ down.T


def attention(h, wq, wk, wo, q_weight, k_weight, sink, heads, kv_heads, scale, window, eps):
    """Causal attention over the last ``window`` tokens, no rotation, a per-head sink in the
    denominator; the raw key projection is also the value."""
    T = h.shape[0]
    d = wq.shape[0] // heads
    q = (h @ wq.T).view(T, heads, d)
    k = (h @ wk.T).view(T, kv_heads, d)
    v = k
    q = rms_norm(q, q_weight, eps)
    k = rms_norm(k, k_weight, eps)
    out = torch.zeros(T, heads, d, dtype=h.dtype)
    for i in range(T):
        lo = max(0, i - window + 1)
        for hd in range(heads):
            g = hd // (heads // kv_heads)
            s = (k[lo:i + 1, g] @ q[i, hd]) * scale
            m = torch.maximum(s.max(), sink[hd])
            p = torch.exp(s - m)
            out[i, hd] = (p @ v[lo:i + 1, g]) / (p.sum() + torch.exp(sink[hd] - m))
    return out.reshape(T, heads * d) @ wo.T


def causal_conv(x, w, b):
    """Per-channel convolution over time: y[t] = b + sum_k w[:, taps-1-k] x[t-k]."""
    taps = w.shape[1]
    y = b.expand_as(x).clone()
    for k in range(taps):
        if k < x.shape[0]:
            y[k:] += x[:x.shape[0] - k] * w[:, taps - 1 - k]
    return y


def silu(x):
    return x / (1 + torch.exp(-x))


def softplus(x):
    return torch.where(x > 30, x, torch.log1p(torch.exp(torch.clamp(x, max=30))))


def selective_scan(x, dt, A_log, B, C, D, state=None):
    """S[c, n] <- exp(-dt e^{A_log}) S + dt x B;  y = S . C + D x.  Returns (y, S)."""
    A = -torch.exp(A_log)
    S = torch.zeros_like(A) if state is None else state.clone()
    y = torch.empty_like(x)
    for t in range(x.shape[0]):
        S = torch.exp(dt[t][:, None] * A) * S + (dt[t] * x[t])[:, None] * B[t][None, :]
        y[t] = S @ C[t] + D * x[t]
    return y, S


def mamba1(h, w, inner, state, dt_rank):
    """``w``: the mixer's tensors by their short names (in, conv, conv.b, x, dt, dt.b, A_log, D, o)."""
    xz = h @ w["in"].T
    x, z = xz[:, :inner], xz[:, inner:]
    x = silu(causal_conv(x, w["conv"], w["conv.b"]))
    p = x @ w["x"].T
    r, B, C = p[:, :dt_rank], p[:, dt_rank:dt_rank + state], p[:, dt_rank + state:]
    dt = softplus(r @ w["dt"].T + w["dt.b"])
    y, _ = selective_scan(x, dt, w["A_log"], B, C, w["D"])
    return (y * silu(z)) @ w["o"].T


def runs_of(n_layers, loop):
    """Layer index of every run, and whether the embedding output is added ahead of it."""
    lo, hi, times = (loop["start"], loop["stop"], loop["times"]) if loop else (0, 0, 1)
    if hi <= lo:
        return [(i, False) for i in range(n_layers)]
    out = [(i, False) for i in range(lo)]
    for p in range(times):
        out += [(i, p > 0 and i == lo) for i in range(lo, hi)]
    return out + [(i, False) for i in range(hi, n_layers)]


def mix(i, h, cfg, w):
    L = cfg["layers"][i]
    m = L["mixer"]
    t = {k[len(f"l{i}.mix."):]: v for k, v in w.items() if k.startswith(f"l{i}.mix.")}
    if L["type"] == "attention":
        return attention(h, t["q"], t["k"], t["o"], t["q.norm"], t["k.norm"], t["sink"], m["heads"], m["kv_heads"],
                         m["scale"], m["mask"]["size"], cfg["norm"]["eps"])
    return mamba1(h, t, m["inner"], m["state"], m["dt_rank"])


def forward(cfg, weights, tokens, dtype=torch.float64, residuals=None):
    """logits [T, vocab]; ``residuals``: a list that receives the stream after every layer run."""
    w = {k: v.to(dtype) for k, v in weights.items()}
    eps = cfg["norm"]["eps"]
    x = embed(w["embed"], torch.as_tensor(tokens, dtype=torch.long), cfg["embedding"]["scale"])
    x0 = x
    for i, again in runs_of(len(cfg["layers"]), cfg.get("loop")):
        if again:
            x = x + x0
        x = x + rms_norm(mix(i, rms_norm(x, w[f"l{i}.norm1"], eps), cfg, w), w[f"l{i}.norm1b"], eps)
        if cfg["layers"][i].get("mlp"):
            h = rms_norm(x, w[f"l{i}.norm2"], eps)
            x = x + rms_norm(feed_forward(h, w[f"l{i}.mlp.up"], w[f"l{i}.mlp.down"]), w[f"l{i}.norm2b"], eps)
        if residuals is not None:
            residuals.append(x)
    return rms_norm(x, w["final.norm"], eps) @ w["head"].T


def random_weights(cfg, seed=0, dtype=torch.float32):
    """Random weights of the tensors ``cfg`` names, sized so that every mechanism matters."""
    g = torch.Generator().manual_seed(seed)

    def nrm(*shape, s=1.0):
        return torch.randn(*shape, generator=g) * s

    def ones(n):
        return 1.0 + 0.2 * nrm(n)

    W, V = cfg["width"], cfg["vocab"]
    w = {"embed": nrm(V, W), "head": nrm(V, W, s=1 / math.sqrt(W)), "final.norm": ones(W)}
    for i, L in enumerate(cfg["layers"]):
        p, m = f"l{i}.", L["mixer"]
        w[p + "norm1"], w[p + "norm1b"] = ones(W), ones(W)
        if L["type"] == "attention":
            H, G, d = m["heads"], m["kv_heads"], m["dim"]
            w.update({p + "mix.q": nrm(H * d, W, s=W ** -0.5), p + "mix.k": nrm(G * d, W, s=W ** -0.5),
                      p + "mix.o": nrm(W, H * d, s=(H * d) ** -0.5), p + "mix.q.norm": ones(d),
                      p + "mix.k.norm": ones(d), p + "mix.sink": nrm(H)})
        else:
            C, N, R, K = m["inner"], m["state"], m["dt_rank"], m["conv"]
            w.update({p + "mix.in": nrm(2 * C, W, s=W ** -0.5), p + "mix.conv": nrm(C, K, s=K ** -0.5),
                      p + "mix.conv.b": nrm(C, s=0.1), p + "mix.x": nrm(R + 2 * N, C, s=C ** -0.5),
                      p + "mix.dt": nrm(C, R, s=R ** -0.5), p + "mix.dt.b": nrm(C, s=0.5) - 2.0,
                      p + "mix.A_log": torch.rand(C, N, generator=g) * 3 - 1.5, p + "mix.D": nrm(C),
                      p + "mix.o": nrm(W, C, s=C ** -0.5)})
        if L.get("mlp"):
            F = L["mlp"]["ff"]
            w.update({p + "norm2": ones(W), p + "norm2b": ones(W), p + "mlp.up": nrm(F, W, s=W ** -0.5),
                      p + "mlp.down": nrm(W, F, s=F ** -0.5)})
    return {k: v.to(torch.bfloat16).to(dtype) for k, v in w.items()}
