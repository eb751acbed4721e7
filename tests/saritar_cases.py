"""Shared bodies of the Saritar / hybrid-decoder tests: every case takes the device (and the
dtype where it matters), so the CPU suite runs the reference operators and the GPU suite the
HIP kernels against the same plain oracle (tests/saritar_oracle.py)."""
from __future__ import annotations

import math

import torch

import saritar_oracle as O
from docqa_amd import ops
from docqa_amd.engine.kv_cache import StatePool
from docqa_amd.engine.llm_engine import LLMEngine, SamplingParams
from docqa_amd.engine.scheduler import ContinuousEngine
from docqa_amd.engine.trace import TraceReplay
from docqa_amd.models import saritar
from docqa_amd.models.hybrid import HybridModel

F32, BF16 = torch.float32, torch.bfloat16


# ------------------------------------------------------------------ configurations
def att(heads, kv, dim, scale, window, ff=None):
    return {"type": "attention", "mixer": {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": dim, "scale": scale,
                                           "mask": {"size": window}},
            "mlp": {"kind": "dense", "ff": ff} if ff else None}


def ssm(inner, state, dt_rank, conv, ff=None):
    return {"type": "mamba1", "mixer": {"inner": inner, "state": state, "dt_rank": dt_rank, "conv": conv},
            "mlp": {"kind": "dense", "ff": ff} if ff else None}


def conf(width, vocab, layers, loop=None, scale=1.0, eps=1e-5):
    return {"architecture": "Saritar", "vocab": vocab, "width": width, "embedding": {"scale": scale},
            "norm": {"eps": eps}, "layers": layers, "loop": loop}


CONFIGS = {
    # recurrent and attention layers, a loop over both kinds, feed-forwards on both
    "mixed": conf(48, 97, [ssm(72, 5, 3, 4), att(4, 2, 16, 0.3, 9, 40), ssm(56, 8, 7, 3, 24), att(3, 1, 24, 0.2, 17)],
                  {"start": 1, "stop": 3, "times": 3}, 1.7, 1e-4),
    # no loop, multi-head attention (a KV head per query head), odd sizes
    "plain": conf(36, 50, [att(3, 3, 12, 0.5, 6, 20), ssm(30, 3, 2, 2)], None, 0.6, 1e-5),
    # the loop is one pass; a window of one token; one-tap convolution; single state
    "ones": conf(40, 61, [ssm(32, 1, 1, 1), att(2, 1, 8, 1.0, 1)], {"start": 0, "stop": 2, "times": 1}),
    # the loop is the last layer; windows past a block; wide state; many taps
    "edge": conf(64, 80, [att(5, 1, 32, 0.25, 70, 96), ssm(64, 40, 20, 6)], {"start": 1, "stop": 2, "times": 2}, 2.0),
    "recurrent": conf(32, 48, [ssm(48, 16, 4, 4), ssm(48, 16, 4, 4)], {"start": 0, "stop": 1, "times": 2}),
    "attention": conf(32, 48, [att(2, 2, 16, 0.4, 5, 32), att(4, 1, 8, 0.4, 40)], None),
}


def make(name, device, dtype=F32, seed=0, tweak=None):
    js = CONFIGS[name] if isinstance(name, str) else name
    w = O.random_weights(js, seed)
    if tweak:
        tweak(w)
    return js, w, HybridModel(saritar.config_from_json(js), device=device, dtype=dtype, weights=w)


def engine(model, tokens=1024, bs=16, slots=4, **kw):
    kw = dict(dict(max_batch=slots, max_context=tokens, block_size=bs, num_blocks=tokens // bs, use_graphs=False,
                   state_slots=slots), **kw)
    return LLMEngine(model, **kw)


def toks(n, vocab, seed):
    return torch.randint(0, vocab, (n,), generator=torch.Generator().manual_seed(seed)).tolist()


def close(a, b, dtype=F32, what=""):
    """fp32: rounding only; bf16: the error of bf16 activations through a few layers."""
    a, b = a.float().cpu(), b.float()
    d = (a - b).pow(2).mean(-1).sqrt() / b.pow(2).mean().sqrt().clamp(min=1e-3)
    tol = 1e-4 if dtype == F32 else 0.06
    assert torch.isfinite(a).all() and d.max() < tol, (what, float(d.max()), int(d.argmax()))


# ------------------------------------------------------------------ norms, activations
def norm_case(device):
    g = torch.Generator().manual_seed(1)
    for H, rows, S, add in ((30, 3, 1, False), (48, 5, 2, True), (1000, 2, 3, True), (4096, 2, 4, False), (5120, 1, 1, True)):
        eps = 1e-3
        P = torch.randn(S, rows, H, generator=g)
        res, emb = torch.randn(rows, H, generator=g), torch.randn(rows, H, generator=g)
        wp, wn = torch.randn(H, generator=g), torch.randn(H, generator=g)
        x = res + O.rms_norm(P.sum(0), wp, eps) + (emb if add else 0)
        for P_ in (P, P[0]) if S == 1 else (P,):
            r = res.clone().to(device)
            y = ops.sandwich_rmsnorm(P_.to(device), r, wp.to(device), wn.to(device), eps, emb.to(device) if add else None, F32)
            close(r, x, what="residual")
            close(y, O.rms_norm(x, wn, eps), what="norm")
            yb = ops.sandwich_rmsnorm(P_.to(device), res.clone().to(device), wp.to(device), wn.to(device), eps,
                                      emb.to(device) if add else None, BF16)
            assert yb.dtype == BF16
            close(yb, O.rms_norm(x, wn, eps), BF16)
        # tiny rows: eps inside the root decides
        r = torch.zeros(rows, H, device=device)
        y = ops.sandwich_rmsnorm((P * 1e-4).to(device), r, wp.to(device), wn.to(device), eps, None, F32)
        x = O.rms_norm(P.sum(0) * 1e-4, wp, eps)
        close(r, x)
        close(y, O.rms_norm(x, wn, eps))


def embed_case(device):
    g = torch.Generator().manual_seed(2)
    for H, V in ((30, 11), (256, 40)):
        tab, w = torch.randn(V, H, generator=g), torch.randn(H, generator=g)
        ids = torch.tensor([0, V - 1, 3, 3], dtype=torch.int32)
        h = O.embed(tab, ids.long(), 2.5)
        for keep in (True, False):
            r, e, x = ops.embed_scale_rmsnorm(ids.to(device), tab.to(device), 2.5, w.to(device), 1e-5, keep)
            close(r, h)
            close(x, O.rms_norm(h, w, 1e-5))
            assert (e is None) == (not keep)
            if keep:
                assert torch.equal(e, r) and e.data_ptr() != r.data_ptr()


def squared_relu_case(device):
    P = torch.randn(3, 5, 24, generator=torch.Generator().manual_seed(3))
    for p in (P, P[0], P[:, :, :7].contiguous()):
        want = O.squared_relu(p.sum(0) if p.dim() == 3 else p)
        close(ops.squared_relu(p.to(device), F32), want)
        close(ops.squared_relu(p.to(device), BF16), want, BF16)


def relu2_linear_case(device, shapes):
    for M, N, K in shapes:
        g = torch.Generator().manual_seed(M)
        x, w = (torch.randn(n, K, generator=g).to(BF16) for n in (M, N))
        want = O.squared_relu((x.to(device).float() @ w.to(device).float().T / K ** 0.5).cpu())
        for decode in (True, False):
            got = ops.relu2_linear(x.to(device), (w.float() / K ** 0.5).to(BF16).to(device), decode)
            assert got.shape == (M, N) and got.dtype == BF16
            close(got, want, BF16, (M, N, K, decode))


def slab_columns_case(device):
    P = torch.randn(3, 7, 40, generator=torch.Generator().manual_seed(3))
    for p in (P, P[0].contiguous()):
        want = p.sum(0) if p.dim() == 3 else p
        for dt in (F32, BF16):
            a, b = ops.slab_columns(p.to(device), 12, 20, dt)
            assert a.is_contiguous() and b.is_contiguous() and a.dtype == b.dtype == dt
            close(a, want[:, :12], dt)
            close(b, want[:, 12:32], dt)


# ------------------------------------------------------------------ attention
def _paged(T, G, d, bs, device, dtype, seed):
    nb = (T + bs - 1) // bs + 3
    perm = torch.randperm(nb, generator=torch.Generator().manual_seed(seed))[: (T + bs - 1) // bs].to(torch.int32)
    kc = torch.full((nb, G, bs, d), 7.0, dtype=dtype, device=device)      # stale rows of earlier owners
    ks = torch.full((nb, G, bs), 3.0, device=device)
    slots = torch.tensor([int(perm[t // bs]) * bs + t % bs for t in range(T)], dtype=torch.int32, device=device)
    return perm[None].to(device).contiguous(), kc, ks, slots


def _attend(device, dtype, T, H, G, d, bs, window, scale, cuts, sink, qk=None, seed=0):
    """Attention output [T, H d] of one sequence fed in portions ``cuts`` through the cache
    (a portion of one token past the start: the decode form), and the oracle's."""
    eps = 1e-5
    g = torch.Generator().manual_seed(seed)
    qw, kw = 1 + 0.3 * torch.randn(d, generator=g), 1 + 0.3 * torch.randn(d, generator=g)
    qk = torch.randn(T, (H + G) * d, generator=g) if qk is None else qk
    qk = qk.to(dtype).float()
    eye = torch.eye((H + G) * d)
    want = O.attention(qk, eye[:H * d], eye[H * d:], torch.eye(H * d), qw, kw, sink, H, G, scale, window, eps)
    bt, kc, ks, slots = _paged(T, G, d, bs, device, dtype, seed)
    out, t0 = [], 0
    for n in cuts:
        i32 = lambda *v: torch.tensor(v, dtype=torch.int32, device=device)  # noqa: E731
        q = ops.qk_norm_store(qk[t0:t0 + n].to(device, dtype), (qw * kw).to(device), slots[t0:t0 + n], kc, ks, H, eps)
        a = dict(window=window, sink=sink.to(device), k_scale=ks)
        if n == 1 and t0 > 0:
            out.append(ops.window_attn(q, kc, bt, i32(t0 + 1), scale, **a))
        else:
            out.append(ops.window_attn(q, kc, bt, i32(t0), scale, cu=i32(0, n), max_q=n, **a))
        t0 += n
    assert t0 == T
    return torch.cat(out), want


def attention_case(device, dtype):
    for T, H, G, d, bs, window in ((23, 3, 3, 8, 16, 5), (40, 5, 1, 16, 16, 1), (70, 4, 2, 40, 64, 33),
                                   (150, 8, 2, 64, 64, 64), (140, 6, 2, 32, 16, 65), (90, 4, 4, 96, 64, 200),
                                   (131, 8, 1, 128, 64, 100), (66, 20, 1, 48, 32, 40), (50, 2, 1, 256, 64, 30)):
        sink = torch.randn(H, generator=torch.Generator().manual_seed(T)) * 2
        for cuts in ([T], [2, 1, T - 3], [T - 6, 1, 1, 1, 1, 1, 1], [7, 1, 9, 2, T - 19]):
            got, want = _attend(device, dtype, T, H, G, d, bs, window, 0.7 * d ** -0.5, cuts, sink, seed=T)
            close(got, want, dtype, (T, H, G, d, bs, window, cuts))


def window_edge_case(device, dtype):
    """One key outshines all others: a query sees it at distance window - 1 and not at
    distance window, as a prompt's portion and decoded."""
    H, G, d = 4, 2, 32
    for window, j in ((8, 0), (8, 13), (64, 63), (65, 64), (70, 1)):
        T = j + window + 3
        g = torch.Generator().manual_seed(window)
        qk = torch.randn(T, (H + G) * d, generator=g) * 0.1
        star = torch.zeros(d)
        star[0] = 10.0
        qk[:, :H * d] += star.repeat(H)                      # every query looks for the star
        qk[j, H * d:] = star.repeat(G)
        sink = torch.full((H,), -3.0)
        for cuts in ([T], [j + 1, *([1] * (T - j - 1))], [j + 1, window - 2, 2, T - j - 1 - window]):
            cuts = [c for c in cuts if c > 0]
            got, want = _attend(device, dtype, T, H, G, d, 16, window, 6.0, cuts, sink, qk, seed=window)
            close(got, want, dtype, (window, j, cuts))
            seen = want[:, 0]                                # the star's value dominates where it is seen
            assert seen[j + window - 1] > 5 and seen[j + window] < 5
            a = got.float().cpu()[:, 0]
            assert a[j + window - 1] > 5 and a[j + window] < 5


def sink_case(device, dtype):
    """A dominant sink takes the weight (outputs shrink), a negligible one none; the first
    token attends to itself and the sink only."""
    for v in (-30.0, 0.0, 4.0, 12.0):
        sink = torch.tensor([v, -v])
        for cuts in ([20], [1, 1, 18], [18, 1, 1]):
            got, want = _attend(device, dtype, 20, 2, 1, 16, 16, 7, 0.3, cuts, sink, seed=5)
            close(got, want, dtype, (v, cuts))
    got, want = _attend(device, dtype, 1, 2, 1, 16, 16, 7, 0.3, [1], torch.tensor([3.0, 30.0]), seed=6)
    close(got, want, dtype)
    assert want[0, 16:].abs().max() < 1e-6


def general_attention_case(device, dtype):
    """The operator without its options: no window, no sink, no key scale, separate values."""
    g = torch.Generator().manual_seed(9)
    for T, H, G, d, bs in ((37, 4, 2, 32, 16), (75, 4, 1, 128, 64)):
        q = torch.randn(T, H * d, generator=g).to(dtype)
        k, v = (torch.randn(T, G, d, generator=g).to(dtype) for _ in range(2))
        bt, kc, ks, slots = _paged(T, G, d, bs, device, dtype, 4)
        vc = torch.zeros_like(kc)
        for t in range(T):
            kc[slots[t] // bs, :, slots[t] % bs] = k[t].to(device)
            vc[slots[t] // bs, :, slots[t] % bs] = v[t].to(device)
        s = torch.einsum("thd,shd->hts", q.float().view(T, H, d), k.float().repeat_interleave(H // G, 1)) * 0.2
        s = s.masked_fill(torch.ones(T, T, dtype=torch.bool).triu(1), -math.inf)
        want = torch.einsum("hts,shd->thd", torch.softmax(s, -1), v.float().repeat_interleave(H // G, 1)).reshape(T, H * d)
        i32 = lambda *x: torch.tensor(x, dtype=torch.int32, device=device)  # noqa: E731
        close(ops.window_attn(q.to(device), kc, bt, i32(0), 0.2, v_cache=vc, cu=i32(0, T), max_q=T), want, dtype)
        close(ops.window_attn(q[-1:].to(device), kc, bt, i32(T), 0.2, v_cache=vc), want[-1:], dtype)


def batch_attention_case(device, dtype):
    """Packed sequences of unequal length and padded decode rows against each alone."""
    H, G, d, bs, window = 4, 2, 32, 16, 12
    lens, ctx0 = [1, 33, 17, 2], [20, 0, 5, 40]
    g = torch.Generator().manual_seed(11)
    nb = 24
    kc = torch.randn(nb, G, bs, d, generator=g).to(device, dtype)
    ks = (torch.rand(nb, G, bs, generator=g) + 0.5).to(device)
    bt = torch.randperm(nb, generator=g)[:20].view(4, 5).to(torch.int32).to(device)
    q = torch.randn(sum(lens), H * d, generator=g).to(device, dtype)
    sink = torch.randn(H, generator=g).to(device)
    i32 = lambda *x: torch.tensor(x, dtype=torch.int32, device=device)  # noqa: E731
    cu = [0]
    for n in lens:
        cu.append(cu[-1] + n)
    kw = dict(window=window, sink=sink, k_scale=ks)
    both = ops.window_attn(q, kc, bt, i32(*ctx0), 0.2, cu=i32(*cu), max_q=max(lens), **kw)
    for b, n in enumerate(lens):
        one = ops.window_attn(q[cu[b]:cu[b + 1]], kc, bt[b:b + 1].contiguous(), i32(ctx0[b]), 0.2, cu=i32(0, n), max_q=n, **kw)
        close(both[cu[b]:cu[b + 1]], one.cpu(), dtype)
    dec = ops.window_attn(q[:4].contiguous(), kc, bt, i32(21, 0, 80, 1), 0.2, **kw)
    assert torch.equal(dec[1].float().cpu(), torch.zeros(H * d))           # a padded row
    for b, n in ((0, 21), (2, 80), (3, 1)):
        one = ops.window_attn(q[b:b + 1].contiguous(), kc, bt[b:b + 1].contiguous(), i32(n), 0.2, **kw)
        close(dec[b:b + 1], one.cpu(), dtype)


# ------------------------------------------------------------------ recurrent mixers
def _cuts(T):
    return ([T], [2] * (T // 2) + [1] * (T % 2), [1] * T, [T - 3, 1, 2], [5, 2, T - 7])


def conv_case(device, dtype):
    for C, taps, T in ((40, 4, 21), (7, 2, 9), (64, 1, 12), (24, 3, 70), (16, 7, 15)):
        g = torch.Generator().manual_seed(C)
        x = torch.randn(T, 2 * C, generator=g).to(dtype)
        w, b = torch.randn(C, taps, generator=g), torch.randn(C, generator=g)
        want = O.silu(O.causal_conv(x[:, :C].float(), w, b))
        wt, bd = w.t().contiguous().to(device), b.to(device)
        for cuts in _cuts(T):
            for step in (False, True):                      # single tokens: prefill form / decode form
                state = torch.full((3, taps - 1, C), 9.0, dtype=dtype, device=device)   # a former owner's
                i32 = lambda *v: torch.tensor(v, dtype=torch.int32, device=device)  # noqa: E731
                out, t0 = [], 0
                for n in cuts:
                    xs = x[t0:t0 + n].to(device)
                    if n == 1 and step:
                        y, z = ops.conv_step(xs, wt, bd, state, i32(1), i32(t0))
                        close(z, x[t0:t0 + 1, C:].float(), dtype)
                    else:
                        y = ops.causal_conv(xs, wt, bd, state, i32(1), i32(0, n), i32(t0), n)
                    out.append(y)
                    t0 += n
                close(torch.cat(out), want, dtype, (C, taps, T, cuts, step))
                assert (state[0] == 9).all() and (state[2] == 9).all()


def scan_case(device, dtype, sizes=((24, 5, 40), (7, 1, 33), (70, 16, 130), (40, 24, 75), (12, 33, 20), (9, 70, 18),
                                    (5, 130, 9))):
    for C, N, T in sizes:
        g = torch.Generator().manual_seed(C + N)
        Np = (N + 3) // 4 * 4
        x, z = torch.randn(T, C, generator=g).to(dtype), torch.randn(T, C, generator=g).to(dtype)
        dt = (torch.randn(T, C, generator=g) * 2 - 1).to(dtype)
        ld = 3 + 2 * N + 2
        bc = torch.randn(T, ld, generator=g).to(dtype)
        A_log, D, dtb = torch.rand(C, N, generator=g) * 3 - 2, torch.randn(C, generator=g), torch.randn(C, generator=g) * 0.5
        yw, Sw = O.selective_scan(x.double(), O.softplus(dt.double() + dtb.double()), A_log.double(),
                                  bc[:, 3:3 + N].double(), bc[:, 3 + N:3 + 2 * N].double(), D.double())
        want = (yw * O.silu(z.double())).float()
        A2 = torch.zeros(C, Np)
        A2[:, :N] = -torch.exp(A_log) / math.log(2)
        dev = [t.to(device) for t in (A2, D, dtb)]
        for cuts, chunk in [(c, 0) for c in _cuts(T)] + [([T], 16), ([T - 5, 5], 7)]:
            state = torch.full((2, C, Np), 5.0, device=device)
            i32 = lambda *v: torch.tensor(v, dtype=torch.int32, device=device)  # noqa: E731
            out, t0 = [], 0
            for n in cuts:
                sl = slice(t0, t0 + n)
                a = (x[sl].to(device), dt[sl].to(device), bc[sl].to(device), 3, 3 + N, N, z[sl].to(device), *dev, state, i32(1))
                if n == 1 and t0 > 0:
                    out.append(ops.selective_step(*a, i32(t0)))
                else:
                    out.append(ops.selective_scan(*a, i32(0, n), i32(t0), n, chunk))
                t0 += n
            close(torch.cat(out), want, dtype, (C, N, T, cuts, chunk))
            close(state[1, :, :N], Sw.float(), F32, "state")     # fp32 whatever the activations are
            assert (state[0] == 5).all()


def scan_batch_case(device, dtype):
    """Unequal packed sequences, some carried, some new, one without a slot; decode rows of
    more than one workgroup, padded rows leaving state alone."""
    C, N, Np = 40, 8, 8
    g = torch.Generator().manual_seed(3)
    lens, ctx, slots = [3, 90, 1, 17], [0, 12, 4, 0], [2, 0, 3, -1]
    T = sum(lens)
    x, z, dt = (torch.randn(T, C, generator=g).to(device, dtype) for _ in range(3))
    bc = torch.randn(T, 2 * N, generator=g).to(device, dtype)
    par = [t.to(device) for t in (-torch.rand(C, Np, generator=g) * 3, torch.randn(C, generator=g), torch.randn(C, generator=g))]
    S0 = torch.randn(4, C, Np, generator=g).to(device)
    i32 = lambda *v: torch.tensor(v, dtype=torch.int32, device=device)  # noqa: E731
    cu = [0]
    for n in lens:
        cu.append(cu[-1] + n)
    S = S0.clone()
    both = ops.selective_scan(x, dt, bc, 0, N, N, z, *par, S, i32(*slots), i32(*cu), i32(*ctx), max(lens), 32)
    for b, n in enumerate(lens):
        S1, sl = S0.clone(), slice(cu[b], cu[b + 1])
        one = ops.selective_scan(x[sl], dt[sl], bc[sl], 0, N, N, z[sl], *par, S1, i32(slots[b]), i32(0, n), i32(ctx[b]), n, 1000)
        close(both[sl], one.cpu(), dtype)
        if slots[b] >= 0:
            close(S[slots[b]], S1[slots[b]].cpu(), F32)
    assert torch.equal(S[1], S0[1])
    B = 11
    slots = [5, -1, 0, 7, 1, 2, 3, 4, 6, -1, 8]
    S0 = torch.randn(9, C, Np, generator=g).to(device)
    S, pos = S0.clone(), [4] * 10 + [0]
    a = (x[:B], dt[:B], bc[:B], 0, N, N, z[:B], *par)
    y = ops.selective_step(*a, S, i32(*slots), i32(*pos))
    # the step projection inside the step, over more channels and ranks than one MFMA tile
    R, w = 64, torch.randn(C, 64, generator=g).to(device, dtype) * 0.1
    r = torch.randn(B, R, generator=g).to(device, dtype)
    S2, S3 = S0.clone(), S0.clone()
    wd = (r.float() @ w.float().T)
    y2 = ops.selective_step(x[:B], (r, w), *a[2:], S2, i32(*slots), i32(*pos))
    y3 = ops.selective_step(x[:B].float(), wd, *[t.float() if torch.is_tensor(t) else t for t in a[2:]], S3, i32(*slots), i32(*pos))
    close(y2, y3.cpu(), dtype, "fused step projection")
    close(S2, S3.cpu(), F32)
    for r in range(B):
        S1 = S0.clone()
        a1 = tuple(t[r:r + 1].contiguous() if torch.is_tensor(t) and t.dim() == 2 and t.shape[0] == B else t for t in a)
        close(y[r:r + 1], ops.selective_step(*a1, S1, i32(slots[r]), i32(pos[r])).cpu(), dtype)
        if slots[r] >= 0:
            close(S[slots[r]], S1[slots[r]].cpu(), F32)


# ------------------------------------------------------------------ whole models
def run_steps(eng, steps):
    """Feed [(id, tokens)] batches through the engine's trace replay; all logits by id."""
    tr, out = TraceReplay(eng), {}
    for step in steps:
        res = tr.step([{"id": i, "tokens": t, "want": list(range(len(t)))} for i, t in step])
        k = 0
        for i, t in step:
            out.setdefault(i, []).append(res[k:k + len(t)])
            k += len(t)
    for i in list(tr.live):
        tr.finish(i)
    return {i: torch.cat(v) for i, v in out.items()}


def portions(seq, sizes):
    out, t = [], 0
    for n in sizes:
        out.append(seq[t:t + n])
        t += n
    return [p for p in out + [seq[t:]] if p]


def whole_case(name, device, dtype, T=45):
    js, w, m = make(name, device, dtype)
    seq = toks(T, js["vocab"], 1)
    res = []
    want = O.forward(js, w, seq, residuals=res)
    m.tap = []
    got = run_steps(engine(m), [[("a", seq)]])["a"]
    assert len(m.tap) == len(res) == len(O.runs_of(len(js["layers"]), js["loop"]))
    for i, (a, b) in enumerate(zip(m.tap, res)):
        close(a, b, dtype, f"run {i}")
    m.tap = None
    close(got, want, dtype, name)


def portions_case(name, device, dtype, T=61):
    js, w, m = make(name, device, dtype, seed=2)
    seq = toks(T, js["vocab"], 3)
    want = O.forward(js, w, seq)
    for sizes in ([2] * 30, [1] * T, [T - 8] + [1] * 8, [16, 16, 16], [15, 2, 17, 3, 1, 1, 9], [3, 1, 2, 31]):
        got = run_steps(engine(m), [[("a", p)] for p in portions(seq, sizes)])["a"]
        close(got, want, dtype, (name, sizes))


def batch_case(name, device, dtype):
    """Requests of unequal length, portions beside decoded tokens, one left out for a while,
    pages and slots given back and taken again, against the oracle on each alone."""
    js, w, m = make(name, device, dtype, seed=4)
    eng = engine(m, tokens=160, bs=16, slots=3)
    V = js["vocab"]
    seqs = {"a": toks(50, V, 5), "b": toks(33, V, 6), "c": toks(9, V, 7), "d": toks(47, V, 8), "e": toks(1, V, 9)}
    want = {k: O.forward(js, w, s) for k, s in seqs.items()}
    at = dict.fromkeys(seqs, 0)
    got = {k: [] for k in seqs}
    tr = TraceReplay(eng)
    plan = [{"a": 20, "b": 1}, {"a": 1, "b": 2, "c": 5}, {"a": 1, "c": 1}, {"b": 16, "c": 1, "a": 1}, {"c": 2, "a": 13},
            {"b": 1, "a": 1, "d": 18}, {"b": 13, "d": 1}, {"d": 2, "a": 13, "e": 1}, {"d": 26}]
    for step in plan:
        es = [{"id": k, "tokens": seqs[k][at[k]:at[k] + n], "want": list(range(n))} for k, n in step.items()]
        out = tr.step(es)
        r = 0
        for k, n in step.items():
            got[k].append(out[r:r + n])
            r += n
            at[k] += n
            if at[k] == len(seqs[k]):
                tr.finish(k)
    assert at == {k: len(s) for k, s in seqs.items()} and not tr.live
    assert eng.kv.allocator.num_free() == 10 and (eng.state is None or eng.state.num_free() == 3)
    for k in seqs:
        close(torch.cat(got[k]), want[k], dtype, (name, k))


def long_decode_case(name, device, dtype, T=150):
    js, w, m = make(name, device, dtype, seed=6)
    seq = toks(T, js["vocab"], 10)
    got = run_steps(engine(m, bs=64), [[("a", p)] for p in portions(seq, [3] + [1] * (T - 3))])["a"]
    close(got, O.forward(js, w, seq), dtype, name)


def far_case(device, dtype):
    """A state that hardly decays carries the first tokens to the end: another first token
    changes the last logits, across portions and decoding."""
    js = conf(32, 40, [ssm(48, 8, 4, 4), att(2, 1, 16, 0.3, 6)], {"start": 0, "stop": 1, "times": 2})

    def slow(w):
        w["l0.mix.A_log"].fill_(-7.0)
        w["l0.mix.dt.b"].fill_(1.0)

    js, w, m = make(js, device, dtype, seed=8, tweak=slow)
    seq = toks(120, 40, 12)
    other = [(seq[0] + 7) % 40] + seq[1:]
    for s in (seq, other):
        want = O.forward(js, w, s)
        for sizes in ([120], [2, 50, 64, 1, 1, 1, 1], [1] * 120):
            close(run_steps(engine(m), [[("a", p)] for p in portions(s, sizes)])["a"], want, dtype, sizes)
    diff = O.forward(js, w, seq)[-1] - O.forward(js, w, other)[-1]
    assert diff.pow(2).mean().sqrt() > 0.01, diff.abs().max()      # 100 x the fp32 tolerance


# ------------------------------------------------------------------ generation
def greedy_oracle(js, w, prompt, n):
    s = list(prompt)
    for _ in range(n):
        s.append(int(O.forward(js, w, s, F32)[-1].argmax()))
    return s[len(prompt):]


def generate_case(name, device, use_graphs=False):
    """Greedy generation through the static engine and the continuous scheduler: chunked
    prefill, several batches, slots and blocks all given back."""
    js, w, m = make(name, device, F32, seed=20)
    V = js["vocab"]
    prompts = [toks(n, V, 30 + n) for n in (1, 5, 40, 19, 33)]
    sp = SamplingParams(max_new_tokens=7)
    want = [greedy_oracle(js, w, p, 7) for p in prompts]
    eng = engine(m, tokens=512, bs=16, slots=8, use_graphs=use_graphs, max_prefill_tokens=24)
    assert eng.generate(prompts, sp) == want
    assert eng.generate(prompts[:2], SamplingParams(max_new_tokens=7, temperature=0.9, top_k=1)) == want[:2]
    ce = ContinuousEngine(engine(m, tokens=512, bs=16, slots=3, use_graphs=use_graphs))
    assert ce.generate(prompts, sp) == want
    for e in (eng, ce.eng):
        assert e.kv.allocator.num_free() == 32 and (e.state is None or e.state.num_free() == e.state.slots)


def mixed_steps_case(name, device):
    """Stall-free admission: prompt chunks ride in decode steps; the tokens do not change."""
    js, w, m = make(name, device, F32, seed=21)
    prompts = [toks(n, js["vocab"], 50 + n) for n in (4, 45, 20, 37)]
    ce = ContinuousEngine(engine(m, tokens=512, bs=16, slots=4))
    ce.mixed, ce.chunk_tokens = True, 16
    futs = [ce.submit(prompts[0], SamplingParams(max_new_tokens=12))]
    for _ in range(3):
        ce.step()
    futs += [ce.submit(p, SamplingParams(max_new_tokens=6)) for p in prompts[1:]]
    while not all(f.done() for f in futs):
        ce.step()
    assert ce.mixed_steps > 0
    for i, (f, p) in enumerate(zip(futs, prompts)):
        assert f.result() == greedy_oracle(js, w, p, 12 if i == 0 else 6)
    assert ce.eng.state is None or ce.eng.state.num_free() == 4


def preemption_case(name, device):
    """The pool runs dry mid-decode: the youngest request loses its blocks and its state slot
    and is computed again from its first token."""
    js, w, m = make(name, device, F32, seed=22)
    prompts = [toks(n, js["vocab"], 70 + n) for n in (15, 14, 13)]
    ce = ContinuousEngine(engine(m, tokens=64, bs=16, slots=3))
    ce.reserve_ahead = 1
    out = ce.generate(prompts, SamplingParams(max_new_tokens=20))
    assert ce.preempted > 0
    assert out == [greedy_oracle(js, w, p, 20) for p in prompts]
    assert ce.eng.kv.allocator.num_free() == 4 and ce.eng.state.num_free() == 3


def state_pool_case():
    pool = StatePool([], 2, "cpu", F32)
    a = pool.alloc(2)
    assert sorted(a) == [0, 1] and pool.num_free() == 0
    for bad in (lambda: pool.alloc(1), ):
        try:
            bad()
            raise AssertionError("expected MemoryError")
        except MemoryError:
            pass
    pool.free([a[0]])
    try:
        pool.free([a[0]])
        raise AssertionError("expected RuntimeError")
    except RuntimeError:
        pass
    assert pool.alloc(1) == [a[0]]
