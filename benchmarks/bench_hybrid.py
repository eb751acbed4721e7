"""Prefill and decode throughput of a hybrid decoder (models/hybrid.py, Saritar layers) at
sizes of real models' layers, beside a Llama decoder of equal width and depth, and the time
of every kernel against its roofline.  Random weights, synthetic token ids.

Run through ``python bench.py --arch saritar`` (one JSON line per row).
"""
from __future__ import annotations

import json
import time

import torch

HBM = 8.0e12            # B/s
MFMA = 2.5e15           # dense bf16 FLOP/s
# fp32 vector issue, the scan's bound: 256 CUs x 4 SIMDs x 16 lanes x 2.4 GHz lane-operations / s;
# a transcendental takes a SIMD's transcendental unit for 8 lanes / clock
LANE_OPS = 256 * 4 * 16 * 2.4e9

# width, inner, state, dt_rank, heads, kv heads, head dim, window, feed-forward
SIZES = {"2b": (2048, 4096, 16, 128, 16, 4, 128, 1024, 8192),
         "8b": (4096, 8192, 16, 256, 32, 8, 128, 1024, 14336)}
LAYERS = 8              # per model: two repeats of [scan, scan, attention + ff, scan]
VOCAB = 32000


def hybrid_config(size: str):
    from docqa_amd.models.hybrid import HybridConfig, LayerSpec, SelectiveScanSpec, WindowAttentionSpec

    W, C, N, R, H, G, d, win, F = SIZES[size]
    ssm = LayerSpec(SelectiveScanSpec(C, N, R, 4))
    att = LayerSpec(WindowAttentionSpec(H, G, d, d ** -0.5, win), F)
    return HybridConfig(name=f"saritar-{size}-layers", vocab_size=VOCAB, hidden=W,
                        layer_specs=[ssm, ssm, att, ssm] * (LAYERS // 4))


def llama_config(size: str):
    from docqa_amd.models.llama import LlamaConfig

    W, _, _, _, H, G, d, _, F = SIZES[size]
    return LlamaConfig(name=f"llama-{size}-layers", vocab_size=VOCAB, hidden=W, intermediate=F, layers=LAYERS, heads=H,
                       kv_heads=G, head_dim=d, bos_token_id=1, eos_token_id=2)


def _engine(model, batch: int, context: int):
    from docqa_amd.engine.llm_engine import LLMEngine

    return LLMEngine(model, max_batch=batch, max_context=context, prefix_cache=False, state_slots=batch,
                     max_prefill_tokens=1 << 20)


def build_model(kind: str, size: str):
    from docqa_amd.models.hybrid import HybridModel
    from docqa_amd.models.llama import LlamaModel

    return HybridModel(hybrid_config(size)) if kind == "saritar" else LlamaModel(llama_config(size))


def bench_model(kind: str, size: str, warmup: int, steps: int, build=build_model) -> list[dict]:
    from docqa_amd.engine.llm_engine import SamplingParams

    model = build(kind, size)
    params = model.cfg.num_params()
    rows = []
    g = torch.Generator().manual_seed(1)
    # prefill: prompts of several lengths, one forward each; decode: graph-replayed steps
    for n, L in ((1, 512), (1, 4096), (16, 512)):
        eng = _engine(model, n, L + 64)
        prompts = torch.randint(0, VOCAB, (n, L), generator=g).tolist()
        sp = SamplingParams(max_new_tokens=1, stop_on_eos=False)
        ts = []
        for i in range(warmup + steps):
            s0 = eng.stats.prefill_s
            eng.generate(prompts, sp)
            if i >= warmup:
                ts.append(eng.stats.prefill_s - s0)
        rows.append({"model": kind, "size": size, "phase": "prefill", "batch": n, "tokens": n * L,
                     "ms": round(1e3 * min(ts), 3), "tokens_per_s": round(n * L / min(ts))})
    for n in (1, 64, 256):
        ctx, gen = 1024, 65
        eng = _engine(model, n, ctx + 2 * gen)
        prompts = torch.randint(0, VOCAB, (n, ctx), generator=g).tolist()
        sp = SamplingParams(max_new_tokens=gen, stop_on_eos=False)
        ts = []
        for i in range(1 + max(1, steps // 2)):
            s0 = eng.stats.decode_s
            eng.generate(prompts, sp)
            if i:
                ts.append((eng.stats.decode_s - s0) / (gen - 1))
        rows.append({"model": kind, "size": size, "phase": "decode", "batch": n, "context": ctx,
                     "ms": round(1e3 * min(ts), 4), "tokens_per_s": round(n / min(ts))})
    for r in rows:
        r["params_M"] = round(params / 1e6)
    del model
    torch.cuda.empty_cache()
    return rows


def _time(fn, iters: int = 20) -> float:
    """Seconds per call, from a graph of ``iters`` calls (no launch gaps)."""
    for _ in range(3):
        fn(0)
    torch.cuda.synchronize()
    graph = torch.cuda.CUDAGraph()
    with torch.cuda.graph(graph):
        for i in range(iters):
            fn(i)
    best = 1e9
    for _ in range(3):
        s, e = torch.cuda.Event(enable_timing=True), torch.cuda.Event(enable_timing=True)
        s.record()
        graph.replay()
        e.record()
        torch.cuda.synchronize()
        best = min(best, s.elapsed_time(e) / iters * 1e-3)
    return best


def bench_kernels(size: str) -> list[dict]:
    """Every kernel of the hybrid decoder and its like in the Llama decoder, alone, against
    its bound: HBM bytes, dense MFMA FLOPs or vector lane-operations, whichever is longest.
    Operands rotate through copies past the 256 MB last-level cache."""
    from docqa_amd import ops

    W, C, N, R, H, G, d, win, F = SIZES[size]
    dev, bf = "cuda", torch.bfloat16
    eps, BS = 1e-5, 64
    out = []

    def rnd(*s, dt=bf):
        return torch.randn(*s, device=dev, dtype=torch.float32).to(dt) if dt != bf else torch.randn(*s, device=dev, dtype=bf)

    def i32(x):
        return torch.as_tensor(x, dtype=torch.int32, device=dev)

    def row(name, phase, M, fn, nbytes=0.0, flops=0.0, lane_ops=0.0, like=""):
        t = _time(fn)
        bound = max(nbytes / HBM, flops / MFMA, lane_ops / LANE_OPS)
        out.append({"kernel": name, "size": size, "phase": phase, "rows": M, "us": round(t * 1e6, 2),
                    "bound_us": round(bound * 1e6, 2), "times_bound": round(t / bound, 2), "like": like})
        torch.cuda.empty_cache()

    def copies(nbytes):
        return max(2, min(16, int(600e6 // max(1, nbytes)) + 1))

    f32 = torch.float32
    wn = torch.ones(W, device=dev)
    A2 = -torch.rand(C, N, device=dev) * 4
    Dv, dtb = torch.ones(C, device=dev), torch.zeros(C, device=dev) - 3
    cw, cb = torch.randn(4, C, device=dev), torch.zeros(C, device=dev)

    for M in (512, 4096):
        nc = copies(M * C * 8)
        res, y = [rnd(M, W, dt=f32) for _ in range(nc)], [rnd(M, W) for _ in range(nc)]
        row("sandwich_rmsnorm", "prefill", M, lambda i: ops.sandwich_rmsnorm(y[i % nc], res[i % nc], wn, wn, eps),
            M * W * (2 + 4 + 4 + 2), like="add_rmsnorm")
        resb, wb = [r.to(bf) for r in res], wn.to(bf)
        row("add_rmsnorm", "prefill", M, lambda i: ops.add_rmsnorm(y[i % nc], resb[i % nc], wb, eps), M * W * 8)
        del res, y, resb
        cu, ctx, sl = i32([0, M]), i32([0]), i32([0])
        xz = [rnd(M, 2 * C) for _ in range(nc)]
        cst = torch.zeros(1, 3, C, device=dev, dtype=bf)
        row("causal_conv", "prefill", M, lambda i: ops.causal_conv(xz[i % nc], cw, cb, cst, sl, cu, ctx, M), M * C * 4,
            like="silu_mul")
        row("silu_mul", "prefill", M, lambda i: ops.silu_mul(xz[i % nc], True), M * C * 6)
        x, dt, bc = [rnd(M, C) for _ in range(nc)], [rnd(M, C) for _ in range(nc)], rnd(M, 2 * N)
        st = torch.zeros(1, C, N, device=dev)
        # a state's step: multiply, exponential (2 lane-operations), two FMAs, multiply
        row("selective_scan", "prefill", M, lambda i: ops.selective_scan(x[i % nc], dt[i % nc], bc, 0, N, N,
                                                                         xz[i % nc][:, C:], A2, Dv, dtb, st, sl, cu, ctx, M),
            M * C * 8, lane_ops=6.0 * M * C * N, like="flash_prefill_paged")
        del xz, x, dt
        nb = (M + BS - 1) // BS
        kc, ks = rnd(nb, G, BS, d), torch.ones(nb, G, BS, device=dev)
        bt, slots = i32([list(range(nb))]), i32(list(range(M)))
        qk, qw = rnd(M, (H + G) * d), torch.ones(d, device=dev)
        row("qk_norm_store", "prefill", M, lambda i: ops.qk_norm_store(qk, qw, slots, kc, ks, H, eps), M * (H + G) * d * 4,
            like="rope_cache")
        qkv = rnd(M, (H + 2 * G) * d)
        kc2, cs = torch.zeros_like(kc), torch.rand(M, d, device=dev)
        row("rope_cache", "prefill", M, lambda i: ops.rope_cache(qkv, slots, cs, slots, kc2, kc2, H, G, d),
            M * ((H + G) * d * 4 + G * d * 6))
        q, sink = rnd(M, H * d), torch.zeros(H, device=dev)
        pairs = sum(min(p + 1, win) for p in range(M))
        row("window_attn", "prefill", M, lambda i: ops.window_attn(q, kc, bt, ctx, d ** -0.5, window=win, sink=sink,
                                                                   k_scale=ks, cu=cu, max_q=M),
            M * (2 * H + G) * d * 2, 4.0 * H * d * pairs, like="flash_prefill_paged")
        row("flash_prefill_paged", "prefill", M, lambda i: ops.flash_prefill_paged(qkv, cu, M, H, G, d, d ** -0.5, kc, kc2,
                                                                                   bt, ctx),
            M * (2 * H + 2 * G) * d * 2, 4.0 * H * d * (M * (M + 1) // 2))
        wu = rnd(F, W)
        xw = rnd(M, W)
        row("relu2_linear", "prefill", M, lambda i: ops.relu2_linear(xw, wu), (F * W + M * (W + F)) * 2, 2.0 * M * F * W,
            like="prefill_glu")
        wg = rnd(2 * F, W)
        row("prefill_glu", "prefill", M, lambda i: ops.prefill_glu(xw, wg), (2 * F * W + M * (W + F)) * 2, 4.0 * M * F * W)
        del wu, wg
        win_, wx, wdt, wo = rnd(2 * C, W), rnd(512 if R + 2 * N > 256 else 256, C), rnd(C, R), rnd(W, C)
        xc = rnd(M, C)
        row("in_proj", "prefill", M, lambda i: ops.linear(xw, win_), (2 * C * W + M * (W + 2 * C)) * 2, 4.0 * M * C * W,
            like="prefill_glu")
        row("x_proj", "prefill", M, lambda i: ops.slab_columns(ops.project(xc, wx), R, 2 * N),
            (wx.numel() + M * (C + R + 2 * N)) * 2, 2.0 * M * (R + 2 * N) * C, like="qkv_proj")
        dti = rnd(M, R)
        row("dt_proj", "prefill", M, lambda i: ops.linear(dti, wdt), (C * R + M * (C + R)) * 2, 2.0 * M * C * R, like="qkv_proj")
        row("out_proj", "prefill", M, lambda i: ops.project(xc, wo), (C * W + M * (C + W)) * 2, 2.0 * M * C * W, like="qkv_proj")
        wq = rnd((H + 2 * G) * d, W)
        row("qkv_proj", "prefill", M, lambda i: ops.project(xw, wq), (wq.numel() + M * (W + wq.shape[0])) * 2, 2.0 * M * wq.numel())

    for B in (1, 64, 256):
        nc = copies(B * C * N * 4)
        sl, pos, ctx = i32(list(range(B))), i32([1024] * B), i32([1025] * B)
        st = [torch.zeros(B, C, N, device=dev) for _ in range(nc)]
        x, z, bc, dti, wdt = rnd(B, C), rnd(B, C), rnd(B, 2 * N), rnd(B, R), rnd(C, R)
        row("selective_step+dt_proj", "decode", B, lambda i: ops.selective_step(x, (dti, wdt), bc, 0, N, N, z, A2, Dv, dtb,
                                                                                st[i % nc], sl, pos),
            B * C * (N * 8 + 6) + C * R * 2, lane_ops=6.0 * B * C * N, like="paged_decode")
        del st
        cst = torch.zeros(B, 3, C, device=dev, dtype=bf)
        P = rnd(B, 2 * C, dt=f32)[None] if B <= 192 else rnd(B, 2 * C)
        row("conv_step", "decode", B, lambda i: ops.conv_step(P, cw, cb, cst, sl, pos),
            B * C * (2 * P.element_size() + 4 + 12), like="rope_cache_splitk")
        nbs = 17
        nc = copies(B * nbs * BS * G * d * 2)
        kcs = [rnd(B * nbs, G, BS, d) for _ in range(nc)]
        ks = torch.ones(B * nbs, G, BS, device=dev)
        bt = i32(torch.arange(B * nbs).view(B, nbs))
        q, sink = rnd(B, H * d), torch.zeros(H, device=dev)
        row("window_attn", "decode", B, lambda i: ops.window_attn(q, kcs[i % nc], bt, ctx, d ** -0.5, window=win, sink=sink,
                                                                  k_scale=ks), B * win * G * (d * 2 + 4), like="paged_decode")
        row("paged_decode", "decode", B, lambda i: ops.paged_decode(q, kcs[i % nc], kcs[(i + 1) % nc], bt, ctx, H, nbs * BS,
                                                                    d ** -0.5), B * 1025 * G * d * 4)
        del kcs
        y, res = rnd(B, W, dt=f32)[None].repeat(4, 1, 1), rnd(B, W, dt=f32)
        row("sandwich_rmsnorm", "decode", B, lambda i: ops.sandwich_rmsnorm(y, res, wn, wn, eps), B * W * (16 + 8 + 2),
            like="add_rmsnorm_splitk")
        resb, wb = res.to(bf), wn.to(bf)
        row("add_rmsnorm_splitk", "decode", B, lambda i: ops.add_rmsnorm_splitk(y, resb, wb, eps), B * W * (16 + 4 + 2))
        qk, kc = rnd(B, (H + G) * d, dt=f32)[None], rnd(B, G, BS, d)
        slots, ks = i32([b * BS for b in range(B)]), torch.ones(B, G, BS, device=dev)
        qw = torch.ones(d, device=dev)
        row("qk_norm_store", "decode", B, lambda i: ops.qk_norm_store(qk, qw, slots, kc, ks, H, eps), B * (H + G) * d * 6,
            like="rope_cache_splitk")
        qkv, cs = rnd(B, (H + 2 * G) * d, dt=f32)[None], torch.rand(2048, d, device=dev)
        kc2 = torch.zeros_like(kc)
        row("rope_cache_splitk", "decode", B, lambda i: ops.rope_cache_splitk(qkv, pos, cs, slots, kc, kc2, H, G, d),
            B * (H + 2 * G) * d * 6)
        for name, n, k, like in (("in_proj", 2 * C, W, "qkv_proj"), ("out_proj", W, C, "qkv_proj"), ("qkv_proj", (H + 2 * G) * d, W, ""),
                                 ("x_proj", 512 if R + 2 * N > 256 else 256, C, "qkv_proj")):
            nc = copies(n * k * 2)
            ws, xx = [rnd(n, k) for _ in range(nc)], rnd(B, k)
            row(name, "decode", B, lambda i: ops.project(xx, ws[i % nc], True), n * k * 2.0, 2.0 * B * n * k, like=like)
            del ws
        nc = copies(F * W * 2)
        ws, xx = [rnd(F, W) for _ in range(nc)], rnd(B, W)
        row("relu2_linear", "decode", B, lambda i: ops.relu2_linear(xx, ws[i % nc], True), F * W * 2.0, 2.0 * B * F * W, like="glu")
        del ws
        ws = [rnd(2 * F, W) for _ in range(nc)]
        cfg = ops.mid_plan(B, 2 * F, W, glu=True)
        glu = (lambda i: ops.gemv_glu(xx, ws[i % nc])) if ops.gemv_glu_ok(B, 2 * F, W) else (
            (lambda i: ops.mgemm_glu(xx, ws[i % nc], cfg[1])) if cfg[0] else (lambda i: ops.glu_linear(xx, ws[i % nc])))
        row("glu", "decode", B, glu, 2.0 * F * W * 2, 4.0 * B * F * W)
        del ws
    return beside_like(out)


def beside_like(out: list[dict]) -> list[dict]:
    """Each kernel's distance from its bound over that of the like kernel (``vs_like``)."""
    at = {(r["kernel"], r["phase"], r["rows"]): r["times_bound"] for r in out}
    for r in out:
        like = at.get((r["like"], r["phase"], r["rows"]))
        if like:
            r["vs_like"] = round(r["times_bound"] / like, 2)
    return out


def main(args, name: str = "saritar", build=build_model, kernels=bench_kernels, beside: tuple = ("llama",)) -> None:
    """Every row of design ``name`` and of the models ``beside`` it, as JSON lines."""
    from docqa_amd import ops

    assert ops.load_native(), ops.native_error()
    torch.set_grad_enabled(False)
    t0 = time.time()
    for size in args.arch_sizes.split(","):
        if args.arch_part in ("all", "models"):
            rows = {}
            for kind in (name, *beside):
                rows[kind] = []
                for r in bench_model(kind, size, args.warmup, args.steps, build):
                    rows[kind].append(r)
                    print(json.dumps(r), flush=True)
            for kind in beside:
                for a, b in zip(rows[name], rows[kind]):
                    print(json.dumps({"size": size, "phase": a["phase"], "batch": a["batch"], "tokens": a.get("tokens", a["batch"]),
                                      f"{name}_over_{kind}": round(a["tokens_per_s"] / b["tokens_per_s"], 2)}), flush=True)
        if args.arch_part in ("all", "kernels"):
            for r in kernels(size):
                print(json.dumps(r), flush=True)
    print(json.dumps({"seconds": round(time.time() - t0, 1)}), flush=True)
