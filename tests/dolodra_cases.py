"""Shared bodies of the Dolodra tests: every case takes the device (and the dtype where it
matters), so the CPU suite runs the reference operators and the GPU suite the HIP kernels
against the same plain oracle (tests/dolodra_oracle.py)."""
from __future__ import annotations

import math

import torch

import dolodra_oracle as O
from docqa_amd import ops
from docqa_amd.engine.llm_engine import SamplingParams
from docqa_amd.engine.scheduler import ContinuousEngine
from docqa_amd.engine.trace import TraceReplay
from docqa_amd.models import dolodra
from docqa_amd.models.hybrid import HybridModel
from saritar_cases import BF16, F32, close, engine, portions, run_steps, toks


# ------------------------------------------------------------------ configurations
def lat(heads, dim, rot, vdim, rank, window, scale=None, base=1e4, ff=None, kv_from=None):
    m = {"heads": heads, "dim": dim, "rot_dim": rot, "vdim": vdim, "kv_rank": rank, "mask": {"size": window},
         "scale": scale or (dim + rot) ** -0.5, "rot": {"base": base, "dims": rot}}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "latent_attention", "mixer": m, "mlp": {"kind": "dense", "ff": ff} if ff else None}


def conf(width, vocab, layers, taps=4, side=8, mult=0.5, cap=20.0, scale=1.0, eps=1e-5):
    return {"architecture": "Dolodra", "vocab": vocab, "width": width, "embedding": {"scale": scale},
            "norm": {"eps": eps}, "residual_mult": mult, "logit_softcap": cap, "canon": {"taps": taps},
            "token_side": {"dim": side}, "layers": layers}


FP32_ONLY = ("sign",)      # rounding flips the sign of an element near zero
CONFIGS = {
    # shared latents with another window and head shape, a layer without feed-forward
    "mixed": conf(48, 97, [lat(4, 16, 8, 24, 40, 9, ff=40), lat(3, 12, 8, 16, 40, 21, ff=24, kv_from=0),
                           lat(2, 24, 16, 8, 32, 17), lat(5, 8, 16, 12, 32, 6, kv_from=2)], 4, 8, 0.6, 9.0, 1.7, 1e-4),
    # nothing a multiple of eight; the source of the latents is not the layer before
    "odd": conf(36, 50, [lat(3, 10, 6, 7, 21, 6, ff=20), lat(2, 5, 2, 9, 13, 40), lat(4, 7, 6, 11, 21, 3, kv_from=0)],
                3, 37, 1.3, 4.0),
    # sizes of one: window, taps, heads, multiplier
    "ones": conf(40, 61, [lat(1, 8, 2, 8, 16, 1, ff=8), lat(1, 1, 2, 1, 16, 33)], 1, 40, 1.0, 30.0),
    # one side element, one latent element: their norms leave a sign
    "sign": conf(40, 61, [lat(2, 8, 2, 8, 16, 12), lat(1, 1, 2, 1, 1, 33)], 3, 1, 0.5, 30.0),
    # windows past a block, many taps, no feed-forward at all, large rotation base
    "edge": conf(64, 80, [lat(6, 32, 16, 32, 64, 70, base=3e5), lat(6, 32, 16, 32, 64, 130, base=3e5, kv_from=0)], 7, 24, 0.4),
    # two readers of one cache, more heads than a row tile
    "readers": conf(32, 48, [lat(20, 8, 8, 8, 48, 40, ff=32), lat(2, 16, 8, 16, 48, 5, ff=32, kv_from=0),
                             lat(1, 8, 8, 24, 48, 64, kv_from=0)], 2, 16, 0.8, 15.0),
}


def make(name, device, dtype=F32, seed=0, tweak=None):
    js = CONFIGS[name] if isinstance(name, str) else name
    w = O.random_weights(js, seed)
    if tweak:
        tweak(w)
    return js, w, HybridModel(dolodra.config_from_json(js), device=device, dtype=dtype, weights=w)


def forms(device, dtype):
    """Expanded or not: the packed operators run on the CPU and as bf16 kernels; fp32 on the GPU
    attends in the latent space only."""
    return (False, True) if device == "cpu" or dtype == BF16 else (False,)


def i32(device, *v):
    return torch.tensor(v, dtype=torch.int32, device=device)


# ------------------------------------------------------------------ stream, activations
def elementwise_case(device):
    g = torch.Generator().manual_seed(1)
    for W, rows, S, S2 in ((30, 3, 1, 1), (48, 5, 2, 3), (1000, 2, 3, 1), (4096, 2, 1, 4)):
        P, Q = torch.randn(S, rows, W, generator=g), torch.randn(S2, rows, W, generator=g)
        res = torch.randn(rows, W, generator=g)
        for q in (Q, None):
            want = res + 0.3 * (P.sum(0) + (q.sum(0) if q is not None else 0))
            for dt in (F32, BF16):
                r = res.clone().to(device)
                out = ops.add_scaled(P.to(device) if S > 1 else P[0].to(device), None if q is None else q.to(device), r, 0.3, dt)
                close(r, want)
                assert out.dtype == dt
                close(out, want, dt)
    P = torch.randn(3, 5, 24, generator=g) * 4
    for p in (P, P[0].contiguous(), P[:, :, :7].contiguous()):
        want = O.gelu_tanh(p.sum(0) if p.dim() == 3 else p)
        close(ops.activation(p.to(device), "gelu_tanh", F32), want)
        close(ops.activation(p.to(device), "gelu_tanh", BF16), want, BF16)
    x = torch.tensor([[-500.0, -30.0, -3.0, 0.0, 1e-3, 7.0, 40.0, 3e4]])
    close(ops.soft_cap(x.to(device), 30.0), O.soft_cap(x, 30.0))
    close(ops.soft_cap(x.to(device, BF16), 5.0), O.soft_cap(x.to(BF16).float(), 5.0))
    z = ops.activation((x * 10).to(device), "gelu_tanh", F32).cpu()
    assert torch.isfinite(z).all() and (z[0, :2] == 0).all() and z[0, 7] == 3e5


def gelu_linear_case(device, shapes):
    for M, N, K in shapes:
        g = torch.Generator().manual_seed(M)
        x, w = (torch.randn(n, K, generator=g).to(BF16) for n in (M, N))
        want = O.gelu_tanh((x.to(device).float() @ w.to(device).float().T / K ** 0.5).cpu())
        for decode in (True, False):
            got = ops.act_linear(x.to(device), (w.float() / K ** 0.5).to(BF16).to(device), "gelu_tanh", decode)
            assert got.shape == (M, N) and got.dtype == BF16
            close(got, want, BF16, (M, N, K, decode))


def side_case(device, dtype):
    """Gate activation times the layer's columns of the token's row, padded columns zero, and the
    product with the projection."""
    for M, n, N, W, S, cols in ((3, 5, 16, 20, 1, 13), (5, 24, 64, 48, 3, 80), (18, 64, 64, 200, 1, 64), (70, 256, 256, 512, 2, 512)):
        g = torch.Generator().manual_seed(n)
        P = torch.randn(S, M, N, generator=g)
        P = P.to(dtype).float() if S == 1 else P
        V = 11
        table = torch.randn(V, cols, generator=g).to(dtype)
        w = (torch.randn(W, N, generator=g) * n ** -0.5).to(dtype)
        ids = torch.randint(0, V, (M,), generator=g, dtype=torch.int32)
        for col in sorted({0, (cols - n) // 8 * 8, cols - n}):
            gate = O.gelu_tanh(P.sum(0)[:, :n]) * table[ids.long(), col:col + n].float()
            p = P.to(device) if S > 1 else P[0].to(device, dtype)
            a = (ids.to(device), table.to(device), col, n)
            got = ops.side_gate(p, *a, dtype)
            close(got[:, :n], gate, dtype, (M, n, N, col))
            assert (got[:, n:] == 0).all()
            close(ops.side_project(p, *a, w.to(device), True), gate @ w[:, :n].float().T, dtype, (M, n, N, W, col))


def norm_conv_case(device, dtype):
    """The stream update, the next norm and its input convolution of one token a row, against the
    three apart, over several steps and with rows that have no slot."""
    for W, taps, S in ((40, 4, 1), (30, 2, 3), (48, 1, 2), (1000, 7, 1)):
        g = torch.Generator().manual_seed(W)
        eps, slots, T = 1e-4, [2, -1, 0], 9
        wp, wn, cw = torch.randn(W, generator=g), torch.randn(W, generator=g), torch.randn(W, taps, generator=g)
        P = torch.randn(T, S, 3, W, generator=g)
        P = P.to(dtype).float() if S == 1 else P
        x = torch.randn(T, 3, W, generator=g)
        conv = cw.t().clone(memory_format=torch.contiguous_format)
        conv[-1] += 1.0
        state = torch.full((3, taps - 1, W), 9.0, dtype=dtype, device=device)
        want_res = x + O.rms(P.sum(1), eps) * wp
        want_h = O.rms(want_res, eps) * wn
        for t in range(T):
            r = x[t].clone().to(device)
            h, hc = ops.sandwich_rmsnorm_conv(P[t].to(device) if S > 1 else P[t, 0].to(device, dtype), r, wp.to(device),
                                              wn.to(device), eps, conv.to(device), state, i32(device, *slots),
                                              i32(device, t, t, t))
            close(r, want_res[t])
            close(h, want_h[t], dtype)
            for b in (0, 2):
                close(hc[b:b + 1], O.conv_input(want_h[:t + 1, b], cw)[t:], dtype, (W, taps, t))
        assert (state[1] == 9).all()


def input_conv_case(device, dtype):
    """h + conv(h) in portions of several sizes, single tokens in both forms; a slot that another
    sequence used; and sequences side by side."""
    from docqa_amd.models.hybrid import InputConv

    for C, taps, T in ((40, 4, 41), (7, 2, 9), (64, 1, 12), (24, 3, 70), (16, 7, 35), (8, 12, 40)):
        g = torch.Generator().manual_seed(C)
        h = torch.randn(T, C, generator=g).to(dtype)
        w = torch.randn(C, taps, generator=g)
        want = O.conv_input(h.float(), w)
        conv = InputConv(w.to(device))
        assert conv.cache_spec().shapes == ((taps - 1, C),)
        for cuts in ([T], [2] * (T // 2) + [1] * (T % 2), [1] * T, [T - 3, 1, 2], [5, 2, T - 7]):
            for step in (False, True):
                state = torch.full((3, taps - 1, C), 9.0, dtype=dtype, device=device)
                out, t0 = [], 0
                for n in cuts:
                    x = h[t0:t0 + n].to(device)
                    if n == 1 and step:
                        out.append(ops.conv_step(x, conv.w, None, state, i32(device, 1), i32(device, t0), silu=False)[0])
                    else:
                        out.append(ops.causal_conv(x, conv.w, None, state, i32(device, 1), i32(device, 0, n),
                                                   i32(device, t0), n, silu=False))
                    t0 += n
                close(torch.cat(out), want, dtype, (C, taps, cuts, step))
                assert (state[0] == 9).all() and (state[2] == 9).all()


# ------------------------------------------------------------------ latent attention
def rope_case(device):
    for r, base, pos in ((2, 10.0, [0, 1, 5]), (16, 1e4, [0, 3, 1000, 99999]), (64, 5e5, list(range(0, 5000, 77)))):
        p = torch.tensor(pos, dtype=torch.int32)
        f = base ** (-torch.arange(0, r, 2, dtype=torch.float64) / r)
        cs = ops.rope_table(p.to(device), f.to(device)).cpu()
        x = torch.zeros(len(pos), r, dtype=torch.float64)
        x[:, :r // 2] = 1.0                                   # the turned unit vectors are (cos, sin)
        assert (cs.double() - O.rotate(x, p, base)).abs().max() < 1e-6


def _rows(T, H, d, r, R, seed):
    """Projection rows [q | latent | key part] and the oracle's view of them: identity weights."""
    g = torch.Generator().manual_seed(seed)
    return torch.randn(T, H * (d + r) + R + r, generator=g)


class Latent:
    """One sequence's latent attention through the operators, in portions, in both forms."""

    def __init__(self, device, dtype, T, H, d, r, vd, R, bs, window, scale, sink, base=1e4, seed=0, rows=None, uk=None, uv=None):
        g = torch.Generator().manual_seed(seed + 1)
        self.device, self.dtype, self.eps = device, dtype, 1e-5
        self.T, self.H, self.d, self.r, self.vd, self.R, self.bs = T, H, d, r, vd, R, bs
        self.window, self.scale, self.base = window, scale, base
        self.sink, self.norm = sink, 1 + 0.3 * torch.randn(R, generator=g)
        self.rows = (_rows(T, H, d, r, R, seed) if rows is None else rows).to(dtype).float()
        self.uk = (torch.randn(H * d, R, generator=g) * R ** -0.5 if uk is None else uk).to(dtype).float()
        self.uv = (torch.randn(H * vd, R, generator=g) * R ** -0.5 if uv is None else uv).to(dtype).float()
        nq = H * (d + r)
        eye = torch.eye(nq + R + r)
        c, kr = O.latent_rows(self.rows, eye[nq:], self.norm, R, base, self.eps)
        self.want = O.latent_attention(self.rows, c, kr, eye[:nq], self.uk, self.uv, torch.eye(H * vd), sink, H, d, vd,
                                       base, scale, window)
        p8 = lambda n: -(-n // 8) * 8  # noqa: E731
        self.d8, self.r8, self.R8, self.v8 = p8(d), p8(r), p8(R), p8(vd)
        pad = torch.nn.functional.pad
        uk, uv = self.uk.view(H, d, R), self.uv.view(H, vd, R)
        up = lambda t: t.to(device, dtype).contiguous()  # noqa: E731
        self.w_qc = up(pad(uk.transpose(1, 2), (0, self.d8 - d, 0, self.R8 - R)))
        self.w_cv = up(pad(uv, (0, self.R8 - R)))
        self.w_kv = up(torch.cat([pad(uk, (0, self.R8 - R, 0, self.d8 - d)).reshape(-1, self.R8),
                                  pad(uv, (0, self.R8 - R, 0, self.v8 - vd)).reshape(-1, self.R8)]))

    def run(self, cuts, expanded=False, slabs=1):
        dev, dt, bs, T = self.device, self.dtype, self.bs, self.T
        nb = (T + bs - 1) // bs
        perm = torch.randperm(nb + 3, generator=torch.Generator().manual_seed(T))[:nb].to(torch.int32)
        cache = torch.full((nb + 3, 1, bs, self.R8 + self.r8), 7.0, dtype=dt, device=dev)      # a former owner's rows
        slots = torch.tensor([int(perm[t // bs]) * bs + t % bs for t in range(T)], dtype=torch.int32, device=dev)
        bt = perm[None].to(dev).contiguous()
        freq = (self.base ** (-torch.arange(0, self.r, 2, dtype=torch.float64) / self.r)).to(dev)
        sink, norm = self.sink.to(dev), self.norm.to(dev)
        out, t0 = [], 0
        for n in cuts:
            x = self.rows[t0:t0 + n]
            if slabs > 1:          # split-K slabs of the projection
                part = torch.randn(slabs - 1, *x.shape, generator=torch.Generator().manual_seed(n))
                P = torch.cat([part, (x - part.sum(0))[None]]).to(dev)
            else:
                P = x.to(dev, dt)
            cs = ops.rope_table(torch.arange(t0, t0 + n, dtype=torch.int32, device=dev), freq)
            q = ops.latent_store(P, cs, slots[t0:t0 + n], cache, norm, self.H, self.d, self.R, self.eps, dt)
            if expanded:
                k0 = max(0, t0 - self.window + 1)
                c, kr = ops.latent_gather(cache, bt, i32(dev, k0), i32(dev, 0, t0 + n - k0), t0 + n - k0, self.R8)
                out.append(ops.packed_window_attn(q, ops.linear(c, self.w_kv), kr, self.H, self.d, self.vd, i32(dev, 0, n),
                                                  i32(dev, 0, t0 + n - k0), n, self.scale, window=self.window, sink=sink))
            else:
                kw = dict(window=self.window, sink=sink)
                q = ops.head_project(q, self.w_qc, self.r8)
                if n == 1 and t0 > 0:
                    out.append(ops.latent_attn(q, cache, bt, i32(dev, t0 + 1), self.scale, self.w_cv, **kw))
                else:
                    out.append(ops.latent_attn(q, cache, bt, i32(dev, t0), self.scale, self.w_cv, cu=i32(dev, 0, n),
                                               max_q=n, **kw))
            t0 += n
        assert t0 == T
        return torch.cat(out)


# T, H, d, r, vd, R, block, window
LATENT_SIZES = ((23, 3, 8, 8, 8, 16, 16, 5), (40, 5, 16, 8, 24, 40, 16, 1), (70, 4, 40, 16, 32, 64, 64, 33),
                (150, 6, 32, 16, 32, 128, 64, 64), (140, 16, 24, 8, 40, 72, 16, 65), (90, 2, 96, 32, 64, 200, 64, 200),
                (131, 9, 128, 64, 128, 256, 64, 100), (200, 20, 64, 32, 96, 512, 32, 150), (70, 40, 16, 64, 16, 96, 64, 70))


def latent_case(device, dtype, sizes=LATENT_SIZES):
    for T, H, d, r, vd, R, bs, window in sizes:
        sink = torch.randn(H, generator=torch.Generator().manual_seed(T)) * 2
        L = Latent(device, dtype, T, H, d, r, vd, R, bs, window, (d + r) ** -0.5, sink, seed=T)
        for k, cuts in enumerate(([T], [2, 1, T - 3], [T - 6, 1, 1, 1, 1, 1, 1], [7, 1, 9, 2, T - 19])):
            close(L.run(cuts, slabs=1 + 2 * (k == 3)), L.want, dtype, (T, H, R, cuts))
            if len(forms(device, dtype)) > 1 and vd % 4 == 0 and L.d8 + L.r8 <= 256:
                close(L.run(cuts, expanded=True), L.want, dtype, ("expanded", T, H, R, cuts))


def latent_odd_case(device, dtype):
    """Sizes that are padded to the kernels' granules, and latents past every MFMA form."""
    for T, H, d, r, vd, R, window in ((30, 3, 10, 6, 7, 21, 6), (26, 2, 5, 2, 9, 13, 40), (20, 1, 1, 2, 1, 1, 7),
                                      (25, 2, 12, 70, 20, 600, 9)):
        sink = torch.randn(H, generator=torch.Generator().manual_seed(T))
        L = Latent(device, dtype, T, H, d, r, vd, R, 16, window, 0.4, sink, seed=T)
        for cuts in ([T], [2, 1, T - 3], [T - 3, 1, 1, 1]):
            close(L.run(cuts), L.want, dtype, (T, H, R, cuts))


def window_edge_case(device, dtype):
    """One latent outshines all others: a query sees it at distance window - 1 and not at distance
    window, as a prompt's portion, decoded, and through packed keys."""
    H, d, r, vd, R = 4, 32, 16, 32, 64
    uk = torch.zeros(H, d, R)
    uk[:, 0, 0] = 1.0
    uv = torch.zeros(H, vd, R)
    uv[:, 0, 0] = 1.0
    for window, j in ((8, 0), (8, 13), (64, 63), (65, 64), (70, 1), (129, 60)):
        T = j + window + 3
        rows = _rows(T, H, d, r, R, window) * 0.1
        lat_at = H * (d + r)
        rows[:, lat_at] = 0.0
        rows[j, lat_at:lat_at + R] = 0.0
        rows[j, lat_at] = 5.0                                # normed: the one large element of its row
        rows[:, :lat_at].view(T, H, d + r)[:, :, 0] = 3.0    # every query looks for it
        L = Latent(device, dtype, T, H, d, r, vd, R, 16, window, 1.0, torch.full((H,), -3.0), seed=window, rows=rows,
                   uk=uk.reshape(H * d, R), uv=uv.reshape(H * vd, R))
        L.norm = torch.ones(R)
        c, kr = O.latent_rows(L.rows, torch.eye(lat_at + R + r)[lat_at:], L.norm, R, L.base, L.eps)
        L.want = O.latent_attention(L.rows, c, kr, torch.eye(lat_at + R + r)[:lat_at], L.uk, L.uv, torch.eye(H * vd), L.sink, H, d, vd,
                                    L.base, L.scale, window)
        seen = L.want[:, 0]
        assert seen[j + window - 1] > 4 and seen[j + window].abs() < 0.1
        for cuts in ([T], [j + 1, *([1] * (T - j - 1))], [j + 1, window - 2, 2, T - j - 1 - window]):
            cuts = [c for c in cuts if c > 0]
            for expanded in forms(device, dtype):
                got = L.run(cuts, expanded)
                close(got, L.want, dtype, (window, j, cuts, expanded))
                a = got.float().cpu()[:, 0]
                assert a[j + window - 1] > 4 and a[j + window].abs() < 0.1, (window, j, cuts, expanded)


def sink_case(device, dtype):
    """A dominant sink takes the weight (outputs shrink), a negligible one none; it is not scaled
    and counts once however the keys are split."""
    for v in (-30.0, 0.0, 4.0, 12.0):
        sink = torch.tensor([v, -v])
        L = Latent(device, dtype, 90, 2, 16, 8, 16, 64, 16, 80, 0.05, sink, seed=5)
        for cuts in ([90], [1, 1, 88], [88, 1, 1]):
            for expanded in forms(device, dtype):
                close(L.run(cuts, expanded), L.want, dtype, (v, cuts, expanded))
    L = Latent(device, dtype, 1, 2, 16, 8, 16, 64, 16, 7, 0.3, torch.tensor([3.0, 30.0]), seed=6)
    close(L.run([1]), L.want, dtype)
    assert L.want[0, 16:].abs().max() < 1e-6


def batch_latent_case(device, dtype):
    """Packed sequences of unequal length and padded decode rows against each alone, in the
    latent space and through packed keys."""
    H, d8, r8, R8, vd, bs, window = 6, 16, 8, 64, 16, 16, 28
    lens, ctx0 = [1, 33, 17, 2], [20, 0, 5, 40]
    g = torch.Generator().manual_seed(11)
    cache = torch.randn(24, 1, bs, R8 + r8, generator=g).to(device, dtype)
    bt = torch.randperm(24, generator=g)[:20].view(4, 5).to(torch.int32).to(device)
    q = torch.randn(sum(lens), H * (R8 + r8), generator=g).to(device, dtype)
    sink = torch.randn(H, generator=g).to(device)
    cu = [0]
    for n in lens:
        cu.append(cu[-1] + n)
    kw = dict(window=window, sink=sink)
    wv = (torch.randn(H, vd, R8, generator=g) * R8 ** -0.5).to(device, dtype)
    both = ops.latent_attn(q, cache, bt, i32(device, *ctx0), 0.1, wv, cu=i32(device, *cu), max_q=max(lens), **kw)
    assert both.shape == (sum(lens), H * vd)
    plain = ops.head_project(ops.window_attn(q, cache, bt, i32(device, *ctx0), 0.1, cu=i32(device, *cu), max_q=max(lens),
                                             v_dim=R8, **kw), wv)
    close(both, plain.cpu(), dtype)
    for b, n in enumerate(lens):
        one = ops.latent_attn(q[cu[b]:cu[b + 1]], cache, bt[b:b + 1].contiguous(), i32(device, ctx0[b]), 0.1, wv,
                              cu=i32(device, 0, n), max_q=n, **kw)
        close(both[cu[b]:cu[b + 1]], one.cpu(), dtype)
    dec = ops.latent_attn(q[:4].contiguous(), cache, bt, i32(device, 21, 0, 80, 1), 0.1, wv, **kw)
    assert torch.equal(dec[1].float().cpu(), torch.zeros(H * vd))           # a padded row
    for b, n in ((0, 21), (2, 80), (3, 1)):
        one = ops.latent_attn(q[b:b + 1].contiguous(), cache, bt[b:b + 1].contiguous(), i32(device, n), 0.1, wv, **kw)
        close(dec[b:b + 1], one.cpu(), dtype)
    if len(forms(device, dtype)) == 1:
        return
    # the visible rows packed
    first = [max(0, c - window + 1) for c in ctx0]
    cuk = [0]
    for c, n, k in zip(ctx0, lens, first):
        cuk.append(cuk[-1] + c + n - k)
    c, kr = ops.latent_gather(cache, bt, i32(device, *first), i32(device, *cuk), cuk[-1], R8)
    flat = cache[bt.long(), 0].flatten(1, 2)
    for b in range(4):
        rows = flat[b, first[b]:ctx0[b] + lens[b]]
        assert torch.equal(c[cuk[b]:cuk[b + 1]], rows[:, :R8]) and torch.equal(kr[cuk[b]:cuk[b + 1]], rows[:, R8:])
    w = (torch.randn(H * (d8 + vd), R8, generator=g) * R8 ** -0.5).to(device, dtype)
    qx = torch.randn(sum(lens), H * (d8 + r8), generator=g).to(device, dtype)
    kv = ops.linear(c, w)
    both = ops.packed_window_attn(qx, kv, kr, H, d8, vd, i32(device, *cu), i32(device, *cuk), max(lens), 0.2, window, sink)
    for b, n in enumerate(lens):
        s = slice(cuk[b], cuk[b + 1])
        one = ops.packed_window_attn(qx[cu[b]:cu[b + 1]], kv[s], kr[s], H, d8, vd, i32(device, 0, n),
                                     i32(device, 0, cuk[b + 1] - cuk[b]), n, 0.2, window, sink)
        close(both[cu[b]:cu[b + 1]], one.cpu(), dtype)


def head_project_case(device, dtype):
    for T, H, K, N, E in ((1, 3, 8, 16, 8), (5, 2, 40, 20, 0), (17, 4, 128, 512, 64), (70, 2, 256, 136, 16), (33, 3, 520, 129, 0),
                          (50, 2, 64, 7, 0), (9, 1, 2048, 64, 0)):
        g = torch.Generator().manual_seed(K)
        x = torch.randn(T, H * (K + E), generator=g).to(dtype)
        w = (torch.randn(H, N, K, generator=g) * K ** -0.5).to(dtype)
        xh = x.float().view(T, H, K + E)
        want = torch.cat([torch.einsum("thk,hnk->thn", xh[..., :K], w.float()), xh[..., K:]], -1).reshape(T, -1)
        close(ops.head_project(x.to(device), w.to(device), E), want, dtype, (T, H, K, N, E))


# ------------------------------------------------------------------ whole models
def whole_case(name, device, dtype, T=45):
    js, w, m = make(name, device, dtype)
    seq = toks(T, js["vocab"], 1)
    res = []
    want = O.forward(js, w, seq, residuals=res)
    m.tap = []
    got = run_steps(engine(m), [[("a", seq)]])["a"]
    assert len(m.tap) == len(res) == len(js["layers"])
    for i, (a, b) in enumerate(zip(m.tap, res)):
        close(a, b, dtype, f"{name}: layer {i}")
    m.tap = None
    close(got, want, dtype, name)
    assert got.dtype == F32 and got.abs().max() <= js["logit_softcap"]


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
    assert eng.kv.allocator.num_free() == 10 and eng.state.num_free() == 3
    for k in seqs:
        close(torch.cat(got[k]), want[k], dtype, (name, k))


def long_decode_case(name, device, dtype, T=150):
    js, w, m = make(name, device, dtype, seed=6)
    seq = toks(T, js["vocab"], 10)
    got = run_steps(engine(m, bs=64), [[("a", p)] for p in portions(seq, [3] + [1] * (T - 3))])["a"]
    close(got, O.forward(js, w, seq), dtype, name)


def far_case(device, dtype):
    """One key far back that outshines the hundreds after it: the token that makes it decides the
    logits as long as it is in the window, and no longer, whatever the portions."""
    window, T, at = 120, 200, 40
    js = conf(32, 40, [lat(2, 8, 8, 16, 24, window), lat(2, 8, 8, 16, 24, window, kv_from=0)], 2, 4, 0.7, 30.0)

    def star(w):
        # token 7 alone has a large first element of its embedding and of its latent; every query
        # looks for it through a constant second element
        w["embed"][:, 0], w["embed"][:, 1] = 0.0, 3.0
        w["embed"][7] = 0.0
        w["embed"][7, 0], w["embed"][7, 1] = 12.0, 3.0
        for i in (0, 1):
            w[f"l{i}.norm1"].zero_()
            w[f"l{i}.canon1"].zero_()
            q = w[f"l{i}.mix.q"].view(2, 16, 32)
            q.mul_(0.1)
            q[:, 0] = 0.0
            q[:, 0, 1] = 4.0
            uk = w[f"l{i}.mix.uk"].view(2, 8, 24)
            uk.mul_(0.2)
            uk[:, 0] = 0.0
            uk[:, 0, 0] = 6.0
            w[f"l{i}.mix.sink"].fill_(-4.0)
        dkv = w["l0.mix.dkv"]
        dkv[0] = 0.0
        dkv[0, 0] = 4.0
        dkv[:, 0][1:] = 0.0
        w["l0.mix.dkv.norm"].fill_(1.0)

    js, w, m = make(js, device, dtype, seed=8, tweak=star)
    seq = [t if t != 7 else 8 for t in toks(T, 40, 12)]
    other, seq = list(seq), list(seq)
    seq[at] = 7
    wa, wb = O.forward(js, w, seq), O.forward(js, w, other)
    gap = (wa - wb).pow(2).mean(-1).sqrt()
    assert gap[at + window - 1] > 0.5 and gap[at + window:].max() < 1e-9
    for sizes in ([T], [2, 50, 64, 1, 1, 1, 1], [at + window - 1] + [1] * (T - at - window + 1), [at + 1] + [1] * (T - at - 1)):
        for s, want in ((seq, wa), (other, wb)):
            close(run_steps(engine(m), [[("a", p)] for p in portions(s, sizes)])["a"], want, dtype, sizes)


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
        assert e.kv.allocator.num_free() == 32 and e.state.num_free() == e.state.slots


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
    assert ce.eng.state.num_free() == 4


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
