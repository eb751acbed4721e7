"""Plain, slow implementation of the Dolodra decoder, one function per mechanism.

Everything runs over whole sequences without a cache, in the dtype of the weights it is
given (the tests use float64).  It shares no code with the package: it is what the product
path is compared against.

Notation: W width, H heads, n / r / v the unrotated, rotated and value sizes of a head, R
the latent size, S the side size.
"""
from __future__ import annotations

import math

import torch


def rms(x, eps):
    """x scaled to unit root mean square over its last axis; eps is added inside the root."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def norm_around_one(x, w, eps):
    """RMS norm whose stored weight is the distance from one."""
    return rms(x, eps) * (1 + w)


def gelu_tanh(z):
    return 0.5 * z * (1 + torch.tanh(math.sqrt(2 / math.pi) * (z + 0.044715 * z ** 3)))


def soft_cap(z, cap):
    return cap * torch.tanh(z / cap)


def embed(table, tokens, scale):
    return table[tokens] * scale


def conv_input(h, w):
    """h plus its causal convolution per channel; the last tap weighs the current token."""
    taps = w.shape[1]
    y = h.clone()
    for back in range(taps):
        if back < h.shape[0]:
            y[back:] += h[:h.shape[0] - back] * w[:, taps - 1 - back]
    return y


def rotate(x, positions, base):
    """x [T, ..., r]: dimension i and i + r/2 turned by position * base^(-2 i / r)."""
    r = x.shape[-1]
    f = torch.tensor([base ** (-2 * i / r) for i in range(r // 2)], dtype=torch.float64)
    a = positions.to(torch.float64)[:, None] * f
    shape = (x.shape[0],) + (1,) * (x.dim() - 2) + (r // 2,)
    c, s = torch.cos(a).to(x.dtype).view(shape), torch.sin(a).to(x.dtype).view(shape)
    u, v = x[..., :r // 2], x[..., r // 2:]
    return torch.cat([u * c - v * s, v * c + u * s], -1)


def latent_rows(h, w_dkv, w_norm, rank, base, eps):
    """(c [T, R] normed latents, key part [T, r] rotated, shared by the heads)."""
    p = h @ w_dkv.T
    return rms(p[:, :rank], eps) * w_norm, rotate(p[:, rank:], torch.arange(h.shape[0]), base)


def latent_attention(h, c, kr, wq, wuk, wuv, wo, sink, heads, dim, vdim, base, scale, window):
    """Causal attention over the last ``window`` tokens; keys and values of every head are
    linear in the latents ``c``, the rotated key part ``kr`` is common to the heads; a number
    per head joins the softmax's denominator."""
    T, r = kr.shape
    q = (h @ wq.T).view(T, heads, dim + r)
    qn, qr = q[..., :dim], rotate(q[..., dim:], torch.arange(T), base)
    k = (c @ wuk.T).view(T, heads, dim)
    v = (c @ wuv.T).view(T, heads, vdim)
    out = torch.zeros(T, heads, vdim, dtype=h.dtype)
    for i in range(T):
        lo = max(0, i - window + 1)
        s = (torch.einsum("khd,hd->hk", k[lo:i + 1], qn[i]) + qr[i] @ kr[lo:i + 1].T) * scale
        m = torch.maximum(s.amax(-1), sink)
        p = torch.exp(s - m[:, None])
        out[i] = torch.einsum("hk,khd->hd", p, v[lo:i + 1]) / (p.sum(-1) + torch.exp(sink - m))[:, None]
    return out.reshape(T, heads * vdim) @ wo.T


def feed_forward(h, up, down):
    return gelu_tanh(h @ up.T) @ down.T


def side_input(x, e, gate, proj, w, eps):
    """What a layer adds for its part ``e`` of the token's side embedding."""
    return rms((gelu_tanh(x @ gate.T) * e) @ proj.T, eps) * w


def forward(cfg, weights, tokens, dtype=torch.float64, residuals=None):
    """logits [T, vocab]; ``residuals``: a list that receives the stream after every layer."""
    w = {k: v.to(dtype) for k, v in weights.items()}
    eps, m, S = cfg["norm"]["eps"], cfg["residual_mult"], cfg["token_side"]["dim"]
    tok = torch.as_tensor(tokens, dtype=torch.long)
    x = embed(w["embed"], tok, cfg["embedding"]["scale"])
    side = w["side.embed"][tok]
    latents = {}
    for i, L in enumerate(cfg["layers"]):
        p, mx = f"l{i}.", L["mixer"]
        t = {k[len(p):]: v for k, v in w.items() if k.startswith(p)}
        h = norm_around_one(x, t["norm1"], eps)
        hm = conv_input(h, t["canon1"])
        base = mx["rot"]["base"]
        src = mx.get("kv_from", i)
        if src == i:
            latents[i] = latent_rows(hm, t["mix.dkv"], t["mix.dkv.norm"], mx["kv_rank"], base, eps)
        y = latent_attention(hm, *latents[src], t["mix.q"], t["mix.uk"], t["mix.uv"], t["mix.o"], t["mix.sink"],
                             mx["heads"], mx["dim"], mx["vdim"], base, mx["scale"], mx["mask"]["size"])
        if L.get("mlp"):
            y = y + feed_forward(h, t["mlp.up"], t["mlp.down"])
        x = x + m * y
        x = x + m * side_input(x, side[:, i * S:(i + 1) * S], t["side.gate"], t["side.proj"], t["side.norm"], eps)
        if residuals is not None:
            residuals.append(x)
    return soft_cap(norm_around_one(x, w["final.norm"], eps) @ w["head"].T, cfg["logit_softcap"])


def random_weights(cfg, seed=0, dtype=torch.float32):
    """Random weights of the tensors ``cfg`` names, sized so that every mechanism matters."""
    g = torch.Generator().manual_seed(seed)

    def nrm(*shape, s=1.0):
        return torch.randn(*shape, generator=g) * s

    W, V, S, n = cfg["width"], cfg["vocab"], cfg["token_side"]["dim"], len(cfg["layers"])
    w = {"embed": nrm(V, W), "side.embed": nrm(V, n * S), "head": nrm(V, W, s=1.5 * W ** -0.5), "final.norm": nrm(W, s=0.2)}
    for i, L in enumerate(cfg["layers"]):
        p, m = f"l{i}.", L["mixer"]
        H, d, r, vd, R = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
        w.update({p + "norm1": nrm(W, s=0.2), p + "canon1": nrm(W, cfg["canon"]["taps"], s=0.4),
                  p + "mix.q": nrm(H * (d + r), W, s=1.5 * W ** -0.5), p + "mix.uk": nrm(H * d, R, s=R ** -0.5),
                  p + "mix.uv": nrm(H * vd, R, s=R ** -0.5), p + "mix.sink": nrm(H),
                  p + "mix.o": nrm(W, H * vd, s=2 * (H * vd) ** -0.5),
                  p + "side.gate": nrm(S, W, s=W ** -0.5), p + "side.proj": nrm(W, S, s=S ** -0.5),
                  p + "side.norm": 1 + nrm(W, s=0.2)})
        if "kv_from" not in m:
            w.update({p + "mix.dkv": nrm(R + r, W, s=W ** -0.5), p + "mix.dkv.norm": 1 + nrm(R, s=0.2)})
        if L.get("mlp"):
            F = L["mlp"]["ff"]
            w.update({p + "mlp.up": nrm(F, W, s=W ** -0.5), p + "mlp.down": nrm(W, F, s=F ** -0.5)})
    return {k: v.to(torch.bfloat16).to(dtype) for k, v in w.items()}
