"""Prefill and decode throughput of a decoder of two-sided and delta mixers with experts
(models/hybrid.py, Gezozen layers) at sizes of real models' layers, beside a Llama decoder of equal
width, depth and active parameters a layer, and the time of every kernel against its roofline.
Random weights, synthetic token ids.

Run through ``python bench.py --arch gezozen`` (one JSON line per row).
"""
from __future__ import annotations

import torch

from . import bench_hybrid as bh
from .bench_hybrid import HBM, LAYERS, MFMA, VOCAB
from .bench_latent import LAUNCH

MFMA32 = 256 * 256 * 2.4e9       # dense fp32 FLOP/s: 256 CUs x 256 / clock x 2.4 GHz

# width, attention heads, their key / value heads, linear-attention heads, delta heads, head dim, window,
# experts, chosen, expert width, shared width (with which a layer's active weights are the Llama's)
SIZES = {"2b": (2048, 8, 2, 8, 16, 128, 1024, 16, 2, 1920, 2048),
         "8b": (4096, 16, 4, 16, 32, 128, 1024, 16, 2, 2816, 4096)}
RANK = 64


def _mixers(size: str):
    from docqa_amd.models.hybrid import AttentionSpec, GatedDeltaSpec, GatedLinearSpec, RetentionSpec, Rotation, TwoSidedSpec

    W, H, G, L, D, d, win, *_ = SIZES[size]
    dec = tuple(1 - 2.0 ** -(5 + 7 * i / (L - 1)) for i in range(L))
    a = TwoSidedSpec(AttentionSpec(H, G, d, d, d ** -0.5, Rotation(5e5, d // 2), 0, 50.0), GatedLinearSpec(L, d, d, 16.0, RANK), 1.0, 1.0)
    b = TwoSidedSpec(AttentionSpec(H, G, d, d, d ** -0.5, Rotation(5e4, d // 2, (8.0, 4096.0, 32.0, 1.0)), win, 0.0, True),
                     RetentionSpec(L, d, d, dec, Rotation(1e6, d)), 1.0, 1.0)
    return a, b, GatedDeltaSpec(D, D // 2, d, d, 4)


def linear_config(size: str):
    from docqa_amd.models.hybrid import HybridConfig, LayerSpec, MoESpec, PostNormForm

    W, *_, E, top, F, Fs = SIZES[size]
    a, b, c = _mixers(size)
    moe = MoESpec(E, top, F, Fs)
    return HybridConfig(name=f"gezozen-{size}-layers", vocab_size=VOCAB, hidden=W, post=PostNormForm(3.0, 4),
                        layer_specs=[LayerSpec(m, moe=moe) for m in (a, b, c, c) * (LAYERS // 4)])


def build_model(kind: str, size: str):
    from docqa_amd.models.hybrid import HybridModel

    return HybridModel(linear_config(size)) if kind == "gezozen" else bh.build_model(kind, size)


def bench_kernels(size: str) -> list[dict]:
    """Every kernel of the decoder and its like in the Llama decoder, alone, against its bound: HBM
    bytes, dense MFMA FLOPs (fp32 ones for the recurrences) or the launch itself, whichever is
    longest.  Operands rotate through copies past the 256 MB last-level cache."""
    from docqa_amd import ops

    W, H, G, L, DH, d, win, E, top, F, Fs = SIZES[size]
    _, _, _, _, HL, GL, dl, _, FL = bh.SIZES[size]
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

    def gemm(name, phase, M, n, k, like="qkv_proj"):
        ws, x = weights(n, k), rnd(M, k)
        row(name, phase, M, lambda i: ops.project(x, ws[i % len(ws)], phase == "decode"),
            (n * k + (M * (k + n) if phase == "prefill" else 0)) * 2.0, 2.0 * M * n * k, like)

    def pad(n):
        return -(-n // 256) * 256

    n_att, n_lin = (H + 2 * G) * d, 4 * L * d
    n_gla, n_del = n_att + n_lin + RANK + W, (2 * (DH // 2) + 2 * DH) * d + 2 * DH + W
    n_moe, n_conv = 2 * Fs + W, (2 * (DH // 2) + DH) * d
    wn, gb, qn = torch.ones(W, device=dev), torch.zeros(W, device=dev), torch.ones(d, device=dev)
    cw = torch.randn(4, n_conv, device=dev)
    freq = (1e4 ** (-torch.arange(0, d // 2, 2, dtype=torch.float64) / (d // 2))).to(dev)
    freq_full = (1e6 ** (-torch.arange(0, d, 2, dtype=torch.float64) / d)).to(dev)

    def mixes():
        """(name, recurrence, decay weights, bias, heads, key heads)"""
        lin = dict(q=n_att, k=n_att + L * d, v=n_att + 2 * L * d, g=n_att + 3 * L * d, a=n_att + 4 * L * d, q_scale=d ** -0.5)
        g = DH * d * 2
        return (("channel", ops.LinearMix("channel", L, L, d, d, rank=RANK, inv_tau=1 / 16, **lin), rnd(L * d, RANK, dt=f32) * 0.1,
                 torch.zeros(L * d, device=dev), n_gla, L),
                ("fixed", ops.LinearMix("fixed", L, L, d, d, **lin), torch.full((L,), -0.01, device=dev), None, n_gla, L),
                ("delta", ops.LinearMix("delta", DH, DH // 2, d, d, 0, DH // 2 * d, DH * d, g, a=g + DH * d, b=g + DH * d + DH, q_scale=d ** -0.5),
                 torch.full((DH,), -1.0, device=dev), torch.zeros(DH, device=dev), n_del, DH))

    for M in (512, 4096):
        ph = "prefill"
        nc = copies(M * W * 8)
        res, y, z = [rnd(M, W, dt=f32) for _ in range(nc)], [rnd(M, W) for _ in range(nc)], rnd(M, W)
        P = rnd(M, pad(n_moe))
        row("post_norm", ph, M, lambda i: ops.post_norm(y[i % nc], z, P, 2 * Fs, gb, res[i % nc], 3.0, wn, 4, eps), M * W * 16,
            like="add_rmsnorm")
        resb, wb = [t.to(bf) for t in res], wn.to(bf)
        row("add_rmsnorm", ph, M, lambda i: ops.add_rmsnorm(y[i % nc], resb[i % nc], wb, eps), M * W * 8)
        del res, y, resb
        cu, ctx, sl, slots = i32([0, M]), i32([0]), i32([0]), i32(list(range(M)))
        nb = (M + BS - 1) // BS
        bt, cs, cs_full = i32([list(range(nb))]), ops.rope_table(slots, freq), ops.rope_table(slots, freq_full)
        kc, vc = rnd(nb, G, BS, d), rnd(nb, G, BS, d)
        P = [rnd(M, pad(n_gla)) for _ in range(copies(M * n_gla * 2))]
        row("qkv_rope_store", ph, M, lambda i: ops.qkv_rope_store(P[i % len(P)], None, qn, qn, cs, slots, kc, vc, H, eps),
            M * (n_att * 4 + d * 2), like="rope_cache")
        q = rnd(M, H * d)
        for name, w, cap in (("attention (cap)", 0, 50.0), ("attention (window)", win, 0.0)):
            pairs = sum(min(p + 1, w or M) for p in range(M))
            row(name, ph, M, lambda i: ops.window_attn(q, kc, bt, ctx, d ** -0.5, window=w, v_cache=vc, cap=cap, cu=cu, max_q=M),
                M * (2 * H + 2 * G) * d * 2, 4.0 * H * d * pairs, like="flash_prefill_paged")
        qkv = [rnd(M, (HL + 2 * GL) * dl) for _ in range(copies(M * HL * dl * 2))]
        kl, kl2, csl = rnd(nb, GL, BS, dl), rnd(nb, GL, BS, dl), torch.rand(M, dl, device=dev)
        row("rope_cache", ph, M, lambda i: ops.rope_cache(qkv[i % len(qkv)], slots, csl, slots, kl, kl2, HL, GL, dl),
            M * ((HL + GL) * dl * 4 + GL * dl * 6))
        row("flash_prefill_paged", ph, M, lambda i: ops.flash_prefill_paged(qkv[0], cu, M, HL, GL, dl, dl ** -0.5, kl, kl2, bt, ctx),
            M * (2 * HL + 2 * GL) * dl * 2, 4.0 * HL * dl * (M * (M + 1) // 2))
        del qkv, P
        for name, mix, wg, b, n, heads in mixes():
            X, st = [rnd(M, pad(n)) for _ in range(copies(M * n * 2))], torch.zeros(1, heads, d, d, device=dev)
            o = rnd(M, heads * d)
            # a head's token: scores of its chunk's earlier half, outputs, state (64 tokens a chunk)
            fl = 2.0 * d * d * 2 + 64 * 2 * d
            if name == "delta":
                fl += 2.0 * d * d + 32 * 2 * d * 3
            row(f"linear_scan ({name})", ph, M, lambda i: ops.linear_scan(X[i % len(X)], X[i % len(X)], mix, wg, b, cs_full if name == "fixed"
                                                                        else None, qn, st, sl, cu, ctx, M, o),
                M * heads * d * 10, M * heads * fl, like="flash_prefill_paged", peak=MFMA32)
            del X
        X = [rnd(M, pad(n_del)) for _ in range(copies(M * n_del * 2))]
        cst = torch.zeros(1, 3, n_conv, device=dev, dtype=bf)
        row("causal_conv", ph, M, lambda i: ops.causal_conv(X[i % len(X)], cw, None, cst, sl, cu, ctx, M), M * n_conv * 4, like="silu_mul")
        g2 = [rnd(M, 2 * FL) for _ in range(copies(M * FL * 6))]
        row("silu_mul", ph, M, lambda i: ops.silu_mul(g2[i % len(g2)], True), M * FL * 6)
        P, sc = [rnd(M, pad(n_moe)) for _ in range(copies(M * n_moe * 2))], torch.ones(M, device=dev)
        row("shared_glu", ph, M, lambda i: ops.glu(P[i % len(P)], 0, Fs, sc), M * Fs * 6, like="silu_mul")
        del X, g2, P
        rw, x = [rnd(E + 1, W) for _ in range(16)], rnd(M, W)
        row("moe_route", ph, M, lambda i: ops.moe_route(x, rw[i % 16], E, top), (M + E) * W * 2, 2.0 * M * W * E, like="qkv_proj")
        ids, wts, _ = ops.moe_route(x, rw[0], E, top)
        up, down = rnd(E, 2, F, W), rnd(E, W, F)
        row("moe_experts", ph, M, lambda i: ops.moe_experts(x, ids, wts, up, down), (E * 3 * F * W + M * top * (W + 3 * F + W)) * 2.0,
            6.0 * M * top * F * W, like="prefill_glu")
        del up, down
        gemm("in_proj (two sides)", ph, M, pad(n_gla), W)
        gemm("in_proj (delta)", ph, M, pad(n_del), W)
        gemm("in_proj (experts)", ph, M, pad(n_moe), W)
        gemm("o_proj", ph, M, W, (H + L) * d)
        gemm("shared_down", ph, M, W, Fs)
        gemm("qkv_proj", ph, M, (HL + 2 * GL) * dl, W, like="")
        ws, x = weights(2 * FL, W), rnd(M, W)
        row("prefill_glu", ph, M, lambda i: ops.prefill_glu(x, ws[i % len(ws)]), (2 * FL * W + M * (W + FL)) * 2.0, 4.0 * M * FL * W)
        del ws

    for B in (1, 64, 256):
        ph = "decode"
        sl, pos, ctx, slots = i32(list(range(B))), i32([1024] * B), i32([1025] * B), i32([b * BS for b in range(B)])
        y, res = rnd(B, W, dt=f32)[None].repeat(4, 1, 1), rnd(B, W, dt=f32)
        P = ops.project(rnd(B, W), rnd(pad(n_gla), W), True)
        S, eb = (P.shape[0] if P.dim() == 3 else 1), P.element_size()
        row("post_norm", ph, B, lambda i: ops.post_norm(y, None, P, n_gla - W, gb, res, 3.0, wn, 4, eps), B * W * (16 + S * eb + 8 + 2),
            like="add_rmsnorm_splitk")
        resb, wb = res.to(bf), wn.to(bf)
        row("add_rmsnorm_splitk", ph, B, lambda i: ops.add_rmsnorm_splitk(y, resb, wb, eps), B * W * (16 + 4 + 2))
        cs = ops.rope_table(pos, freq)
        kc, vc = rnd(B, G, BS, d), rnd(B, G, BS, d)
        row("qkv_rope_store", ph, B, lambda i: ops.qkv_rope_store(P, None, qn, qn, cs, slots, kc, vc, H, eps), B * n_att * (S * eb + 2),
            like="rope_cache_splitk")
        qkv, csl = rnd(B, (HL + 2 * GL) * dl, dt=f32)[None], torch.rand(2048, dl, device=dev)
        kl, kl2 = torch.zeros(B, GL, BS, dl, device=dev, dtype=bf), torch.zeros(B, GL, BS, dl, device=dev, dtype=bf)
        row("rope_cache_splitk", ph, B, lambda i: ops.rope_cache_splitk(qkv, pos, csl, slots, kl, kl2, HL, GL, dl), B * (HL + 2 * GL) * dl * 6)
        nbs = 17
        bt = i32(torch.arange(B * nbs).view(B, nbs))
        kcs = [rnd(B * nbs, G, BS, d) for _ in range(copies(B * nbs * BS * G * d * 2) + 1)]
        q = rnd(B, H * d)
        for name, w, cap in (("attention (cap)", 0, 50.0), ("attention (window)", win, 0.0)):
            row(name, ph, B, lambda i: ops.window_attn(q, kcs[i % len(kcs)], bt, ctx, d ** -0.5, window=w, v_cache=kcs[(i + 1) % len(kcs)], cap=cap),
                B * (w or 1025) * G * d * 4, like="paged_decode")
        kcs = [rnd(B * nbs, GL, BS, dl) for _ in range(copies(B * nbs * BS * GL * dl * 2) + 1)]
        q = rnd(B, HL * dl)
        row("paged_decode", ph, B, lambda i: ops.paged_decode(q, kcs[i % len(kcs)], kcs[(i + 1) % len(kcs)], bt, ctx, HL, nbs * BS, dl ** -0.5),
            B * 1025 * GL * dl * 4)
        del kcs
        cs_full = ops.rope_table(pos, freq_full)
        for name, mix, wg, b, n, heads in mixes():
            X = ops.project(rnd(B, W), rnd(pad(n), W), True)
            st = [torch.zeros(B, heads, d, d, device=dev) for _ in range(copies(B * heads * d * d * 4))]
            o = rnd(B, heads * d)
            S, eb = (X.shape[0] if X.dim() == 3 else 1), X.element_size()
            row(f"linear_step ({name})", ph, B, lambda i: ops.linear_step(X, X, mix, wg, b, cs_full if name == "fixed" else None, qn, st[i % len(st)],
                                                                        sl, pos, o), B * heads * d * (d * 8 + 4 * S * eb + 2), like="paged_decode")
            if name == "delta":
                cst = torch.zeros(B, 3, n_conv, device=dev, dtype=bf)
                row("conv_step", ph, B, lambda i: ops.conv_step(X, cw, None, cst, sl, pos, rest=n - n_conv),
                    B * (n_conv * (S * eb + 2 + 12) + (n - n_conv) * (S * eb + eb)), like="rope_cache_splitk")
            del st
        rw, x = [rnd(E + 1, W) for _ in range(16)], rnd(B, W)
        row("moe_route", ph, B, lambda i: ops.moe_route(x, rw[i % 16], E, top), (B + E) * W * 2, like="qkv_proj")
        ids, wts, _ = ops.moe_route(x, rw[0], E, top)
        seen = len(set(ids.flatten().tolist()))
        ups, downs = [[rnd(*s) for _ in range(copies(seen * F * W * 2 * 3))] for s in ((E, 2, F, W), (E, W, F))]
        row("moe_experts", ph, B, lambda i: ops.moe_experts(x, ids, wts, ups[i % len(ups)], downs[i % len(ups)]), seen * 3 * F * W * 2.0,
            6.0 * B * top * F * W, like="glu")
        del ups, downs
        P, sc = ops.project(x, rnd(pad(n_moe), W), True), torch.ones(B, device=dev)
        S, eb = (P.shape[0] if P.dim() == 3 else 1), P.element_size()
        row("shared_glu", ph, B, lambda i: ops.glu(P, 0, Fs, sc), B * Fs * (2 * S * eb + 2), like="rope_cache_splitk")
        gemm("in_proj (two sides)", ph, B, pad(n_gla), W)
        gemm("in_proj (delta)", ph, B, pad(n_del), W)
        gemm("in_proj (experts)", ph, B, pad(n_moe), W)
        gemm("o_proj", ph, B, W, (H + L) * d)
        gemm("shared_down", ph, B, W, Fs)
        gemm("qkv_proj", ph, B, (HL + 2 * GL) * dl, W, like="")
        ws, x = weights(2 * FL, W), rnd(B, W)
        cfg = ops.mid_plan(B, 2 * FL, W, glu=True)
        glu = (lambda i: ops.gemv_glu(x, ws[i % len(ws)])) if ops.gemv_glu_ok(B, 2 * FL, W) else (
            (lambda i: ops.mgemm_glu(x, ws[i % len(ws)], cfg[1])) if cfg[0] else (lambda i: ops.glu_linear(x, ws[i % len(ws)])))
        row("glu", ph, B, glu, 2.0 * FL * W * 2, 4.0 * B * FL * W)
        del ws
    return bh.beside_like(out)


def main(args) -> None:
    bh.main(args, "gezozen", build_model, bench_kernels)
