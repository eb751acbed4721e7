"""Prefill and decode throughput of a latent-attention decoder (models/hybrid.py, Dolodra layers)
at sizes of real models' layers, beside a Llama decoder of equal width, depth and parameter count
a layer, and the time of every kernel against its roofline.  Random weights, synthetic token ids.

Run through ``python bench.py --arch dolodra`` (one JSON line per row).
"""
from __future__ import annotations

import torch

from . import bench_hybrid as bh
from .bench_hybrid import HBM, LAYERS, MFMA, VOCAB

LAUNCH = 2.1e-6         # a captured launch that does nothing

# width, heads, head dim, rotated dim, value dim, latent, window, side, feed-forward (half again the
# Llama's: two matrices in place of its three)
SIZES = {"2b": (2048, 16, 128, 64, 128, 512, 1024, 256, 12288),
         "8b": (4096, 32, 128, 64, 128, 512, 1024, 256, 21504)}


def latent_config(size: str):
    from docqa_amd.models import dolodra
    from docqa_amd.models.hybrid import LatentAttentionSpec, LayerSpec, ParallelForm

    W, H, d, r, vd, R, win, S, F = SIZES[size]
    layers = [LayerSpec(LatentAttentionSpec(H, d, r, vd, R, (d + r) ** -0.5, win, 1e4, None if i % 2 == 0 else i - 1), F)
              for i in range(LAYERS)]
    return dolodra._config(f"dolodra-{size}-layers", ParallelForm(0.5, 4, S), 30.0, vocab_size=VOCAB, hidden=W,
                           layer_specs=layers, embed_scale=W ** 0.5)


def build_model(kind: str, size: str):
    from docqa_amd.models.hybrid import HybridModel

    return HybridModel(latent_config(size)) if kind == "dolodra" else bh.build_model(kind, size)


def bench_kernels(size: str) -> list[dict]:
    """Every kernel of the latent-attention decoder and its like in the Llama decoder, alone,
    against its bound: HBM bytes, dense MFMA FLOPs or the launch itself, whichever is longest.
    Operands rotate through copies past the 256 MB last-level cache."""
    from docqa_amd import ops

    W, H, d, r, vd, R, win, S, F = SIZES[size]
    _, _, _, _, HL, G, dl, _, FL = bh.SIZES[size]
    D = R + r
    dev, bf, f32 = "cuda", torch.bfloat16, torch.float32
    eps, BS = 1e-5, 64
    out = []

    def rnd(*s, dt=bf):
        return torch.randn(*s, device=dev, dtype=f32).to(dt) if dt != bf else torch.randn(*s, device=dev, dtype=bf)

    def i32(x):
        return torch.as_tensor(x, dtype=torch.int32, device=dev)

    def row(name, phase, M, fn, nbytes=0.0, flops=0.0, like=""):
        t = bh._time(fn)
        bound = max(nbytes / HBM, flops / MFMA, LAUNCH)
        out.append({"kernel": name, "size": size, "phase": phase, "rows": M, "us": round(t * 1e6, 2),
                    "bound_us": round(bound * 1e6, 2), "times_bound": round(t / bound, 2), "like": like})
        torch.cuda.empty_cache()

    def copies(nbytes):
        return max(2, min(16, int(600e6 // max(1, nbytes)) + 1))

    def weights(n, k):
        return [rnd(n, k) for _ in range(copies(n * k * 2))]

    def gemm(name, phase, M, n, k, like="qkv_proj", fn=None, rows=None):
        """A projection of M rows; ``rows``: the useful ones of a padded weight."""
        ws, x = weights(n, k), rnd(M, k)
        m = rows or n
        f = fn or (lambda x, w: ops.project(x, w, phase == "decode"))
        row(name, phase, M, lambda i: f(x, ws[i % len(ws)]), (m * k + (M * (k + m) if phase == "prefill" else 0)) * 2.0,
            2.0 * M * m * k, like)

    def pad(n):
        return -(-n // 256) * 256

    wn, cw = torch.ones(W, device=dev), torch.randn(4, W, device=dev)
    nq = H * (d + r)
    table = rnd(VOCAB, LAYERS * S)
    gelu = lambda dec: (lambda x, w: ops.act_linear(x, w, "gelu_tanh", dec))  # noqa: E731

    for M in (512, 4096):
        ph = "prefill"
        nc = copies(M * W * 8)
        res, y, y2 = [rnd(M, W, dt=f32) for _ in range(nc)], [rnd(M, W) for _ in range(nc)], rnd(M, W)
        row("add_scaled", ph, M, lambda i: ops.add_scaled(y[i % nc], y2, res[i % nc], 0.5), M * W * (4 + 8 + 2), like="add_rmsnorm")
        row("sandwich_rmsnorm", ph, M, lambda i: ops.sandwich_rmsnorm(y[i % nc], res[i % nc], wn, wn, eps), M * W * 12,
            like="add_rmsnorm")
        resb, wb = [t.to(bf) for t in res], wn.to(bf)
        row("add_rmsnorm", ph, M, lambda i: ops.add_rmsnorm(y[i % nc], resb[i % nc], wb, eps), M * W * 8)
        cu, ctx, sl = i32([0, M]), i32([0]), i32([0])
        cst = torch.zeros(1, 3, W, device=dev, dtype=bf)
        row("causal_conv", ph, M, lambda i: ops.causal_conv(y[i % nc], cw, None, cst, sl, cu, ctx, M, silu=False), M * W * 4,
            like="silu_mul")
        g2 = [rnd(M, 2 * FL) for _ in range(copies(M * FL * 6))]
        row("silu_mul", ph, M, lambda i: ops.silu_mul(g2[i % len(g2)], True), M * FL * 6)
        del res, y, resb, g2
        slots, ids = i32(list(range(M))), i32(torch.randint(0, VOCAB, (M,)))
        nb = (M + BS - 1) // BS
        cache, bt = rnd(nb, 1, BS, D), i32([list(range(nb))])
        cs = ops.rope_table(slots, (1e4 ** (-torch.arange(0, r, 2, dtype=torch.float64) / r)).to(dev))
        P = [rnd(M, pad(nq + D)) for _ in range(copies(M * (nq + D) * 4))]
        norm = torch.ones(R, device=dev)
        row("latent_store", ph, M, lambda i: ops.latent_store(P[i % len(P)], cs, slots, cache, norm, H, d, R, eps, bf),
            M * ((nq + D) * 4 + r * 4), like="rope_cache")
        del P
        qkv = [rnd(M, (HL + 2 * G) * dl) for _ in range(copies(M * HL * dl * 2))]
        kc, kc2 = torch.zeros(nb, G, BS, dl, device=dev, dtype=bf), torch.zeros(nb, G, BS, dl, device=dev, dtype=bf)
        csl = torch.rand(M, dl, device=dev)
        row("rope_cache", ph, M, lambda i: ops.rope_cache(qkv[i % len(qkv)], slots, csl, slots, kc, kc2, HL, G, dl),
            M * ((HL + G) * dl * 4 + G * dl * 6))
        row("flash_prefill_paged", ph, M, lambda i: ops.flash_prefill_paged(qkv[0], cu, M, HL, G, dl, dl ** -0.5, kc, kc2, bt, ctx),
            M * (2 * HL + 2 * G) * dl * 2, 4.0 * HL * dl * (M * (M + 1) // 2))
        row("latent_gather", ph, M, lambda i: ops.latent_gather(cache, bt, ctx, cu, M, R), M * D * 4, like="rope_cache")
        q, kv, kr = rnd(M, nq), rnd(M, H * (d + vd)), rnd(M, r)
        sink = torch.zeros(H, device=dev)
        pairs = sum(min(p + 1, win) for p in range(M))
        row("packed_window_attn", ph, M, lambda i: ops.packed_window_attn(q, kv, kr, H, d, vd, cu, cu, M, (d + r) ** -0.5, win, sink),
            M * (nq + H * (d + 2 * vd) + r) * 2, 2.0 * H * (d + r + vd) * pairs, like="flash_prefill_paged")
        qs, kcs = rnd(M, HL * dl), rnd(nb, G, BS, dl)
        row("window_attn", ph, M, lambda i: ops.window_attn(qs, kcs, bt, ctx, dl ** -0.5, window=win, sink=torch.zeros(HL, device=dev),
                                                            cu=cu, max_q=M), M * (2 * HL + G) * dl * 2, 4.0 * HL * dl * pairs)
        gemm("kv_proj", ph, M, H * (d + vd), R, fn=ops.linear)
        gemm("in_proj", ph, M, pad(nq + D), W, rows=nq + D)
        gemm("o_proj", ph, M, W, H * vd)
        gemm("gelu_linear", ph, M, F, W, like="prefill_glu", fn=gelu(False))
        gemm("down_proj", ph, M, W, F)
        gemm("side_gate_proj", ph, M, S, W, fn=ops.narrow_project)
        ws, P = weights(W, S), rnd(M, S)
        row("side_project", ph, M, lambda i: ops.side_project(P, ids, table, 0, S, ws[i % len(ws)]), (W * S + M * (2 * S + W)) * 2.0,
            2.0 * M * W * S, like="qkv_proj")
        gemm("qkv_proj", ph, M, (HL + 2 * G) * dl, W, like="")
        ws, x = weights(2 * FL, W), rnd(M, W)
        row("prefill_glu", ph, M, lambda i: ops.prefill_glu(x, ws[i % len(ws)]), (2 * FL * W + M * (W + FL)) * 2.0, 4.0 * M * FL * W)
        del ws

    for B in (1, 64, 256):
        ph = "decode"
        sl, pos, ctx = i32(list(range(B))), i32([1024] * B), i32([1025] * B)
        ids, slots = i32(torch.randint(0, VOCAB, (B,))), i32([b * BS for b in range(B)])
        y, res = rnd(B, W, dt=f32)[None].repeat(4, 1, 1), rnd(B, W, dt=f32)
        row("add_scaled", ph, B, lambda i: ops.add_scaled(y, y, res, 0.5), B * W * (32 + 8 + 2), like="add_rmsnorm_splitk")
        yb = rnd(B, W)
        resb, wb = res.to(bf), wn.to(bf)
        row("add_rmsnorm_splitk", ph, B, lambda i: ops.add_rmsnorm_splitk(y, resb, wb, eps), B * W * (16 + 4 + 2))
        cst = torch.zeros(B, 3, W, device=dev, dtype=bf)
        row("sandwich_rmsnorm_conv", ph, B, lambda i: ops.sandwich_rmsnorm_conv(yb, res, wn, wn, eps, cw, cst, sl, pos),
            B * W * (2 + 8 + 4 + 12), like="add_rmsnorm_splitk")
        P, cache = rnd(B, pad(nq + D), dt=f32)[None], rnd(B, 1, BS, D)
        cs = ops.rope_table(pos, (1e4 ** (-torch.arange(0, r, 2, dtype=torch.float64) / r)).to(dev))
        norm = torch.ones(R, device=dev)
        row("latent_store", ph, B, lambda i: ops.latent_store(P, cs, slots, cache, norm, H, d, R, eps, bf), B * (nq + D) * 6,
            like="rope_cache_splitk")
        qkv, csl = rnd(B, (HL + 2 * G) * dl, dt=f32)[None], torch.rand(2048, dl, device=dev)
        kc, kc2 = torch.zeros(B, G, BS, dl, device=dev, dtype=bf), torch.zeros(B, G, BS, dl, device=dev, dtype=bf)
        row("rope_cache_splitk", ph, B, lambda i: ops.rope_cache_splitk(qkv, pos, csl, slots, kc, kc2, HL, G, dl),
            B * (HL + 2 * G) * dl * 6)
        nbs = 17
        bt = i32(torch.arange(B * nbs).view(B, nbs))
        caches = [rnd(B * nbs, 1, BS, D) for _ in range(copies(B * nbs * BS * D * 2))]
        qc, sink = rnd(B, H * D), torch.zeros(H, device=dev)
        wv = [rnd(H, vd, R) for _ in range(8)]
        row("latent_attn", ph, B, lambda i: ops.latent_attn(qc, caches[i % len(caches)], bt, ctx, (d + r) ** -0.5, wv[i % 8],
                                                            window=win, sink=sink),
            (B * (win * D + H * (D + vd)) + H * vd * R) * 2.0, 2.0 * B * H * (win * (D + R) + vd * R), like="paged_decode")
        del caches
        kcs = [rnd(B * nbs, G, BS, dl) for _ in range(copies(B * nbs * BS * G * dl * 2))]
        q = rnd(B, HL * dl)
        row("paged_decode", ph, B, lambda i: ops.paged_decode(q, kcs[i % len(kcs)], kcs[(i + 1) % len(kcs)], bt, ctx, HL, nbs * BS,
                                                              dl ** -0.5), B * 1025 * G * dl * 4)
        row("window_attn", ph, B, lambda i: ops.window_attn(q, kcs[i % len(kcs)], bt, ctx, dl ** -0.5, window=win,
                                                            sink=torch.zeros(HL, device=dev)), B * win * G * dl * 2)
        del kcs
        for name, n, k, e in (("absorb_q", R, d, r),):
            ws, x = [rnd(H, n, k) for _ in range(copies(H * n * k * 2))], rnd(B, H * (k + e))
            row(name, ph, B, lambda i: ops.head_project(x, ws[i % len(ws)], e), (H * n * k + B * H * (n + k + 2 * e)) * 2.0,
                2.0 * B * H * n * k, like="qkv_proj")
            del ws
        gemm("in_proj", ph, B, pad(nq + D), W, rows=nq + D)
        gemm("o_proj", ph, B, W, H * vd)
        gemm("gelu_linear", ph, B, F, W, like="glu", fn=gelu(True))
        gemm("down_proj", ph, B, W, F)
        gemm("side_gate_proj", ph, B, S, W)
        P = ops.project(rnd(B, W), rnd(S, W), True)
        ws = weights(W, S)
        row("side_project", ph, B, lambda i: ops.side_project(P, ids, table, 0, S, ws[i % len(ws)], True),
            W * S * 2.0 + B * (S * 4 + S * 2 + W * 2), 2.0 * B * W * S, like="qkv_proj")
        gemm("qkv_proj", ph, B, (HL + 2 * G) * dl, W, like="")
        ws, x = weights(2 * FL, W), rnd(B, W)
        cfg = ops.mid_plan(B, 2 * FL, W, glu=True)
        glu = (lambda i: ops.gemv_glu(x, ws[i % len(ws)])) if ops.gemv_glu_ok(B, 2 * FL, W) else (
            (lambda i: ops.mgemm_glu(x, ws[i % len(ws)], cfg[1])) if cfg[0] else (lambda i: ops.glu_linear(x, ws[i % len(ws)])))
        row("glu", ph, B, glu, 2.0 * FL * W * 2, 4.0 * B * FL * W)
        del ws
    return bh.beside_like(out)


def main(args) -> None:
    bh.main(args, "dolodra", build_model, bench_kernels)
