"""Prefill and decode throughput of a decoder of channel-delta and latent-attention mixers with experts in
groups (models/hybrid.py, Pifazen layers) at sizes of real models' layers, beside the closest other
decoder (Gezozen: delta rule, experts) and a Llama of equal width, depth and active parameters a layer, and
the time of every kernel against its roofline and against the like kernel of the closest decoder that has
one.  Random weights, synthetic token ids.

Run through ``python bench.py --arch pifazen`` (one JSON line per row).
"""
from __future__ import annotations

import torch

from . import bench_hybrid as bh
from . import bench_linear as bl
from .bench_hybrid import HBM, LAYERS, MFMA, VOCAB
from .bench_latent import LAUNCH
from .bench_linear import MFMA32

# width, heads of both mixers, head dim, rotated dim, latent, query latent, inner size of decay and gate, experts,
# identity experts, chosen, groups, kept, expert width, dense width (with which a layer's active weights are the Llama's)
SIZES = {"2b": (2048, 16, 128, 64, 512, 768, 128, 16, 2, 4, 3, 2, 1792, 10240),
         "8b": (4096, 32, 128, 64, 512, 1536, 128, 16, 2, 4, 3, 2, 3072, 18432)}
YARN = (8.0, 4096.0, 32.0, 1.0)


def channel_config(size: str):
    from docqa_amd.models import pifazen
    from docqa_amd.models.hybrid import ChannelDeltaSpec, GroupRouter, LayerSpec, MoESpec

    W, H, d, r, R, Q, K, E, ident, top, groups, keep, F, FD = SIZES[size]
    moe = MoESpec(E, top, F, router=GroupRouter(ident, groups, keep, 2.0), limit=7.0)
    c = LayerSpec(ChannelDeltaSpec(H, H, d, d, 4, K, K), moe=moe)
    a = LayerSpec(pifazen._latent(H, d, r, d, R, (d + r) ** -0.5, 5e5, Q, gate="element"), FD)
    b = LayerSpec(pifazen._latent(H, d, r, d, R, (d + r) ** -0.5, 1e6, scaling=YARN), moe=moe)
    return pifazen._config(f"pifazen-{size}-layers", vocab_size=VOCAB, hidden=W, layer_specs=[c, c, a, b] * (LAYERS // 4))


def build_model(kind: str, size: str):
    from docqa_amd.models.hybrid import HybridModel

    return HybridModel(channel_config(size)) if kind == "pifazen" else bl.build_model(kind, size)


def bench_kernels(size: str) -> list[dict]:
    """Every kernel of the decoder and its like in the closest one, alone, against its bound: HBM bytes, dense
    MFMA FLOPs (fp32 ones for the recurrences) or the launch itself, whichever is longest.  Operands rotate
    through copies past the 256 MB last-level cache."""
    from docqa_amd import ops

    W, H, d, r, R, Q, K, E, ident, top, groups, keep, F, FD = SIZES[size]
    D, nq, n_conv, N = R + r, H * (d + r), 3 * H * d, E + ident
    dev, bf, f32 = "cuda", torch.bfloat16, torch.float32
    eps, BS = 1e-5, 64
    out = []

    def rnd(*s, dt=bf):
        return torch.randn(*s, device=dev, dtype=f32).to(dt) if dt != bf else torch.randn(*s, device=dev, dtype=bf)

    def i32(x):
        return torch.as_tensor(x, dtype=torch.int32, device=dev)

    def row(name, phase, M, fn, nbytes=0.0, flops=0.0, like="", peak=MFMA):
        t = bh._time(fn)
        bound = max(nbytes / HBM, flops / peak, LAUNCH)
        out.append({"kernel": name, "size": size, "phase": phase, "rows": M, "us": round(t * 1e6, 2),
                    "bound_us": round(bound * 1e6, 2), "times_bound": round(t / bound, 2), "like": like})
        torch.cuda.empty_cache()

    def copies(nbytes):
        return max(2, min(16, int(600e6 // max(1, nbytes)) + 1))

    def weights(n, k):
        return [rnd(n, k) for _ in range(copies(n * k * 2))]

    def gemm(name, phase, M, n, k, like="o_proj", fn=None, rows=None):
        """A projection of M rows; ``rows``: the useful ones of a padded weight."""
        ws, x, m = weights(n, k), rnd(M, k), rows or n
        f = fn or (lambda x, w: ops.project(x, w, phase == "decode"))
        row(name, phase, M, lambda i: f(x, ws[i % len(ws)]), (m * k + (M * (k + m) if phase == "prefill" else 0)) * 2.0, 2.0 * M * m * k, like)

    def pad(n):
        return -(-n // 256) * 256

    # rows of the input projections: delta, latent (query latent, gate an element), latent (queries, gate a head)
    n_del, n_lat, n_lat2 = n_conv + 2 * K + H, Q + D + H * d, nq + D + H
    wn, scale, norm, qn = (torch.ones(n, device=dev) for n in (W, W, R, Q))
    hn = torch.ones(d, device=dev)
    freq = (1e4 ** (-torch.arange(0, r, 2, dtype=torch.float64) / r)).to(dev)
    cw = torch.randn(4, n_conv, device=dev)
    wa, wg = rnd(H * d, K), rnd(H * d, K)
    act, fb = torch.full((4,), 0.3, device=dev), torch.zeros(FD, device=dev)
    A, Ab = torch.full((H,), -1.0, device=dev), torch.full((H * d,), -2.0, device=dev)
    mix = ops.LinearMix("channel_delta", H, H, d, d, 0, H * d, 2 * H * d, H * d, a=0, b=2 * H * d, q_scale=d ** -0.5, gate="sigmoid")
    at = 3 * H * d
    mix_delta = ops.LinearMix("delta", H, H, d, d, 0, H * d, 2 * H * d, at, a=at + H * d, b=at + H * d + H, q_scale=d ** -0.5)
    Db = torch.zeros(H, device=dev)
    zw = 2 * H * d + H
    corr = torch.zeros(N, device=dev)

    def experts(ph, M):
        rw, rl, x = [rnd(N, W) * W ** -0.5 for _ in range(16)], [rnd(E + 1, W) for _ in range(16)], rnd(M, W)
        row("moe_route_groups", ph, M, lambda i: ops.moe_route_groups(x, rw[i % 16], corr, top, groups, keep, 2.0), (M + N) * W * 2,
            2.0 * M * W * N, like="moe_route")
        row("moe_route", ph, M, lambda i: ops.moe_route(x, rl[i % 16], E, top), (M + E) * W * 2, 2.0 * M * W * E)
        ids, wts = ops.moe_route_groups(x, rw[0], corr, top, groups, keep, 2.0)
        il, wl, _ = ops.moe_route(x, rl[0], E, top)
        nw = copies(E * F * W * 6) if ph == "decode" else 1
        ups, downs = [[rnd(*s) for _ in range(nw)] for s in ((E, 2, F, W), (E, W, F))]
        for name, i_, w_, limit, like in (("moe_experts (clamped)", ids, wts, 7.0, "moe_experts"), ("moe_experts", il, wl, 0.0, "")):
            real = i_[i_ < E]
            seen, pairs = len(set(real.tolist())), real.numel()
            row(name, ph, M, lambda i: ops.moe_experts(x, i_, w_, ups[i % nw], downs[i % nw], limit),
                seen * 3 * F * W * 2.0 + (pairs * (2 * W + 2 * F) * 2.0 if ph == "prefill" else 0), 6.0 * pairs * F * W, like)

    for M in (512, 4096):
        ph = "prefill"
        nc = copies(M * W * 8)
        res, y = [rnd(M, W, dt=f32) for _ in range(nc)], [rnd(M, W) for _ in range(nc)]
        row("scaled_rmsnorm", ph, M, lambda i: ops.scaled_rmsnorm(y[i % nc], res[i % nc], scale, wn, eps), M * W * 12, like="post_norm")
        ids, wts = i32(torch.randint(0, N, (M, top))), torch.ones(M, top, device=dev)
        ys = [rnd(top, M, W) for _ in range(nc // 2 + 1)]
        row("scaled_rmsnorm (experts)", ph, M, lambda i: ops.scaled_rmsnorm(ys[i % len(ys)], res[i % nc], scale, wn, eps, mix=(ids, wts, E, y[0])),
            M * W * (10 + 2 * top), like="post_norm")
        P, z = rnd(M, W), rnd(M, W)
        row("post_norm", ph, M, lambda i: ops.post_norm(y[i % nc], z, P, 0, wn, res[i % nc], 3.0, wn, 4, eps), M * W * 16)
        del res, y, ys
        cu, ctx, sl, slots = i32([0, M]), i32([0]), i32([0]), i32(list(range(M)))
        nb = (M + BS - 1) // BS
        bt, cs, cache = i32([list(range(nb))]), ops.rope_table(slots, freq), rnd(nb, 1, BS, D)
        P = [rnd(M, pad(n_lat)) for _ in range(copies(M * n_lat * 2))]
        row("latent_norm_store", ph, M, lambda i: ops.latent_norm_store(P[i % len(P)], cs, slots, cache, qn, norm, eps, bf),
            M * ((Q + D) * 4 + r * 4), like="latent_store")
        P = [rnd(M, pad(nq + D)) for _ in range(copies(M * (nq + D) * 4))]
        row("latent_store (queries)", ph, M, lambda i: ops.latent_store(P[i % len(P)], cs, slots, cache, None, H, d, R, eps, bf),
            M * (nq * 4 + r * 4), like="latent_store")
        row("latent_store", ph, M, lambda i: ops.latent_store(P[i % len(P)], cs, slots, cache, norm, H, d, R, eps, bf), M * ((nq + D) * 4 + r * 4))
        del P
        q, kv, kr, sink = rnd(M, nq), rnd(M, 2 * H * d), rnd(M, r), torch.zeros(H, device=dev)
        P = rnd(M, pad(n_lat))
        for name, win, s, gate, like in (("packed_attn (gate an element)", 0, None, (P, Q + D, 1, 0), "packed_window_attn"),
                                         ("packed_attn (gate a head)", 0, None, (P, Q + D, d, 0), "packed_window_attn"),
                                         ("packed_window_attn", 1024, sink, None, "")):
            pairs, ng = sum(min(p + 1, win or M) for p in range(M)), 0 if gate is None else H * d // gate[2]
            row(name, ph, M, lambda i: ops.packed_window_attn(q, kv, kr, H, d, d, cu, cu, M, (d + r) ** -0.5, win, s, gate),
                M * (nq + 3 * H * d + r + ng) * 2, 2.0 * H * (2 * d + r) * pairs, like=like)
        g2, sc = [rnd(M, 2 * H * d) for _ in range(copies(M * H * d * 4))], torch.ones(M, device=dev)
        row("glu", ph, M, lambda i: ops.glu(g2[i % len(g2)], 0, H * d, sc), M * H * d * 6)
        del g2
        P = [rnd(M, FD) for _ in range(copies(M * FD * 4))]
        row("poly_norm", ph, M, lambda i: ops.poly_norm(P[i % len(P)], fb, act, FD, eps), M * FD * 4, like="activation")
        row("activation", ph, M, lambda i: ops.activation(P[i % len(P)], "gelu_tanh"), M * FD * 4)
        del P
        # a head's token: scores of its chunk's earlier half, outputs, state, the solved triangle (64 tokens a chunk)
        fl = 2.0 * d * d * 3 + 64 * 2 * d + 32 * 2 * d * 3
        o, st = rnd(M, H * d), torch.zeros(1, H, d, d, device=dev)
        X, Z = [rnd(M, n_conv) for _ in range(copies(M * n_conv * 2))], [rnd(M, zw, dt=f32) for _ in range(copies(M * zw * 4))]
        row("linear_scan (channel delta)", ph, M, lambda i: ops.linear_scan(X[i % len(X)], Z[i % len(Z)], mix, A, Ab, None, hn, st, sl, cu, ctx, M, o),
            M * H * d * 16, M * H * fl, like="linear_scan (delta)", peak=MFMA32)
        del X, Z
        X = [rnd(M, pad(at + H * d + 2 * H)) for _ in range(copies(M * n_conv * 2))]
        row("linear_scan (delta)", ph, M, lambda i: ops.linear_scan(X[i % len(X)], X[i % len(X)], mix_delta, A, Db, None, hn, st, sl, cu, ctx, M, o),
            M * H * d * 10, M * H * fl, peak=MFMA32)
        P = [rnd(M, pad(n_del)) for _ in range(copies(M * n_del * 2))]
        row("low_rank", ph, M, lambda i: ops.low_rank(P[i % len(P)], n_conv, wa, wg, H), M * zw * 4 + M * 2 * K * 2 + 4 * H * d * K,
            4.0 * M * H * d * K, like="kv_proj")
        cst = torch.zeros(1, 3, n_conv, device=dev, dtype=bf)
        row("causal_conv", ph, M, lambda i: ops.causal_conv(P[i % len(P)], cw, None, cst, sl, cu, ctx, M), M * n_conv * 4, like="glu")
        del X, P
        experts(ph, M)
        gemm("in_proj (delta)", ph, M, pad(n_del), W, rows=n_del)
        gemm("in_proj (latent, gate)", ph, M, pad(n_lat), W, rows=n_lat)
        gemm("in_proj (latent, queries)", ph, M, pad(n_lat2), W, rows=n_lat2)
        gemm("uq_proj", ph, M, nq, Q)
        gemm("kv_proj", ph, M, 2 * H * d, R, fn=ops.linear)
        gemm("dense_up", ph, M, FD, W)
        gemm("dense_down", ph, M, W, FD)
        gemm("o_proj", ph, M, W, H * d, like="")

    for B in (1, 64, 256):
        ph = "decode"
        sl, pos, ctx, slots = i32(list(range(B))), i32([1024] * B), i32([1025] * B), i32([b * BS for b in range(B)])
        y, res = rnd(B, W, dt=f32)[None].repeat(4, 1, 1), rnd(B, W, dt=f32)
        row("scaled_rmsnorm", ph, B, lambda i: ops.scaled_rmsnorm(y, res, scale, wn, eps), B * W * (16 + 8 + 2), like="post_norm")
        ys, h = rnd(top, B, W), rnd(B, W)
        ids, wts = i32(torch.randint(0, N, (B, top))), torch.ones(B, top, device=dev)
        row("scaled_rmsnorm (experts)", ph, B, lambda i: ops.scaled_rmsnorm(ys, res, scale, wn, eps, mix=(ids, wts, E, h)), B * W * (10 + 2 * top),
            like="post_norm")
        row("post_norm", ph, B, lambda i: ops.post_norm(y, None, h, 0, wn, res, 3.0, wn, 4, eps), B * W * (16 + 2 + 8 + 2))
        cs, cache = ops.rope_table(pos, freq), rnd(B, 1, BS, D)
        P = ops.project(rnd(B, W), rnd(pad(n_lat), W), True)
        S, eb = (P.shape[0] if P.dim() == 3 else 1), P.element_size()
        row("latent_norm_store", ph, B, lambda i: ops.latent_norm_store(P, cs, slots, cache, qn, norm, eps, bf), B * (Q + D) * (S * eb + 2),
            like="latent_store")
        gp, ge = P, S * eb
        P, sc = ops.project(rnd(B, W), rnd(2 * H * d, W), True), torch.ones(B, device=dev)
        S, eb = (P.shape[0] if P.dim() == 3 else 1), P.element_size()
        row("glu", ph, B, lambda i: ops.glu(P, 0, H * d, sc), B * H * d * (2 * S * eb + 2))
        P = ops.project(rnd(B, Q), rnd(nq, Q), True)
        S, eb = (P.shape[0] if P.dim() == 3 else 1), P.element_size()
        row("latent_store (queries)", ph, B, lambda i: ops.latent_store(P, cs, slots, cache, None, H, d, R, eps, bf), B * nq * (S * eb + 2), like="latent_store")
        P = ops.project(rnd(B, W), rnd(pad(nq + D), W), True)
        S, eb = (P.shape[0] if P.dim() == 3 else 1), P.element_size()
        row("latent_store", ph, B, lambda i: ops.latent_store(P, cs, slots, cache, norm, H, d, R, eps, bf), B * (nq + D) * (S * eb + 2))
        nbs = 17
        bt = i32(torch.arange(B * nbs).view(B, nbs))
        caches = [rnd(B * nbs, 1, BS, D) for _ in range(copies(B * nbs * BS * D * 2))]
        qc, sink, wv = rnd(B, H * D), torch.zeros(H, device=dev), [rnd(H, d, R) for _ in range(8)]
        for name, win, s, gate, like in (("latent_attn (gate an element)", 0, None, (gp, Q + D, 1, 0), "latent_attn (window)"),
                                         ("latent_attn (gate a head)", 0, None, (gp, Q + D, d, 0), "latent_attn (window)"),
                                         ("latent_attn (window)", 1024, sink, None, "")):
            n, ng = win or 1025, 0 if gate is None else H * d // gate[2]
            row(name, ph, B, lambda i: ops.latent_attn(qc, caches[i % len(caches)], bt, ctx, (d + r) ** -0.5, wv[i % 8], window=win, sink=s, gate=gate),
                (B * (n * D + H * (D + d)) + H * d * R) * 2.0 + B * ng * ge, 2.0 * B * H * (n * (D + R) + d * R), like=like)
        del caches
        ws, x = [rnd(H, R, d) for _ in range(copies(H * R * d * 2))], rnd(B, nq)
        row("absorb_q", ph, B, lambda i: ops.head_project(x, ws[i % len(ws)], r), (H * R * d + B * H * (R + d + 2 * r)) * 2.0, 2.0 * B * H * R * d, like="o_proj")
        del ws
        P = ops.project(rnd(B, W), rnd(FD, W), True)
        S, eb = (P.shape[0] if P.dim() == 3 else 1), P.element_size()
        row("poly_norm", ph, B, lambda i: ops.poly_norm(P, fb, act, FD, eps), B * FD * (S * eb + 2), like="activation")
        row("activation", ph, B, lambda i: ops.activation(P, "gelu_tanh"), B * FD * (S * eb + 2))
        X, Z, o = rnd(B, n_conv), rnd(B, zw, dt=f32), rnd(B, H * d)
        st = [torch.zeros(B, H, d, d, device=dev) for _ in range(copies(B * H * d * d * 4))]
        row("linear_step (channel delta)", ph, B, lambda i: ops.linear_step(X, Z, mix, A, Ab, None, hn, st[i % len(st)], sl, pos, o),
            B * H * d * (d * 8 + 6 + 8 + 2), like="linear_step (delta)")
        X = rnd(B, pad(at + H * d + 2 * H))
        row("linear_step (delta)", ph, B, lambda i: ops.linear_step(X, X, mix_delta, A, Db, None, hn, st[i % len(st)], sl, pos, o),
            B * H * d * (d * 8 + 8 + 2))
        del st
        z, cst = rnd(B, 2 * K + H), torch.zeros(B, 3, n_conv, device=dev, dtype=bf)
        was, wgs = [rnd(H * d, K) for _ in range(16)], [rnd(H * d, K) for _ in range(16)]
        row("low_rank", ph, B, lambda i: ops.low_rank(z, 0, was[i % 16], wgs[i % 16], H), 4 * H * d * K + B * zw * 4, 4.0 * B * H * d * K, like="absorb_q")
        P = ops.project(rnd(B, W), rnd(pad(n_del), W), True)
        S, eb = (P.shape[0] if P.dim() == 3 else 1), P.element_size()
        row("conv_step", ph, B, lambda i: ops.conv_step(P, cw, None, cst, sl, pos, rest=2 * K + H), B * (n_conv * (S * eb + 2 + 12) + (2 * K + H) * (S * eb + eb)),
            like="glu")
        experts(ph, B)
        gemm("in_proj (delta)", ph, B, pad(n_del), W, rows=n_del)
        gemm("in_proj (latent, gate)", ph, B, pad(n_lat), W, rows=n_lat)
        gemm("in_proj (latent, queries)", ph, B, pad(n_lat2), W, rows=n_lat2)
        gemm("uq_proj", ph, B, nq, Q)
        gemm("dense_up", ph, B, FD, W)
        gemm("dense_down", ph, B, W, FD)
        gemm("o_proj", ph, B, W, H * d, like="")
    return bh.beside_like(out)


def main(args) -> None:
    bh.main(args, "pifazen", build_model, bench_kernels, beside=("gezozen", "llama"))
