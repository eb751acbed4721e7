"""Shared bodies of the Gezozen tests: every case takes the device (and the dtype where it
matters), so the CPU suite runs the reference operators and the GPU suite the HIP kernels
against the same plain oracle (tests/gezozen_oracle.py)."""
from __future__ import annotations

import math

import torch

import gezozen_oracle as O
from docqa_amd import ops
from docqa_amd.engine.llm_engine import SamplingParams
from docqa_amd.engine.scheduler import ContinuousEngine
from docqa_amd.engine.trace import TraceReplay
from docqa_amd.models import gezozen
from docqa_amd.models.hybrid import HybridModel, Rotation
from saritar_cases import BF16, F32, close, engine, portions, run_steps, toks

F64 = torch.float64


# ------------------------------------------------------------------ configurations
def moe(experts, top, ff, shared=0):
    m = {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}
    if shared:
        m["shared"] = {"ff": shared}
    return m


def rot(base, dims, scaling=None):
    r = {"base": base, "dims": dims}
    if scaling:
        r["scaling"] = dict(zip(("factor", "original", "fast", "slow"), scaling))
    return r


def left(heads, kv, dim, vdim, r, scale=None, window=0, cap=None):
    m = {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "scale": scale or dim ** -0.5, "rot": r}
    if window:
        m["mask"] = {"size": window}
    if cap:
        m["softcap"] = cap
    return m


def gla(lf, heads, dim, vdim, tau, ls=1.0, rs=1.0, mlp=None):
    return {"type": "parallel", "mixer": {"left": lf, "right": {"heads": heads, "dim": dim, "vdim": vdim, "tau": tau},
                                          "left_scale": ls, "right_scale": rs}, "mlp": mlp}


def ret(lf, dim, vdim, decay, r, ls=1.0, rs=1.0, mlp=None):
    return {"type": "parallel_2", "mixer": {"left": lf, "right": {"heads": len(decay), "dim": dim, "vdim": vdim, "decay": decay, "rot": r},
                                            "left_scale": ls, "right_scale": rs}, "mlp": mlp}


def delta(heads, kv, dim, vdim, conv, mlp=None):
    return {"type": "delta", "mixer": {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "conv": conv}, "mlp": mlp}


def conf(width, vocab, layers, groups, alpha=2.0, eps=1e-5):
    return {"architecture": "Gezozen", "vocab": vocab, "width": width, "postln_alpha": alpha, "norm": {"eps": eps, "groups": groups},
            "layers": layers}


YARN = (4.0, 64.0, 8.0, 0.5)
CONFIGS = {
    # every mixer; two choices a token, with and without a shared expert
    "mixed": conf(64, 97, [gla(left(4, 2, 16, 24, rot(1e4, 8), 0.3, cap=6.0), 3, 16, 24, 4.0, 0.7, 1.2, moe(5, 2, 24, 16)),
                           ret(left(4, 1, 24, 16, rot(2e3, 16, YARN), window=9), 16, 8, [0.9, 0.99], rot(1e5, 12), 1.1, 0.8, moe(4, 1, 32)),
                           delta(4, 2, 16, 24, 4, moe(6, 2, 16, 40))], 4, 2.5, 1e-4),
    # nothing a multiple of eight, layers without a feed-forward, no cap, no window, full rotation
    "odd": conf(36, 50, [delta(3, 1, 10, 7, 3), ret(left(3, 3, 6, 9, rot(50.0, 6), 0.7), 7, 5, [0.5, 0.97, 1.0], rot(30.0, 6), 0.5, 1.5),
                         gla(left(2, 1, 10, 5, rot(100.0, 2), 0.9, 5, 3.0), 2, 9, 3, 2.0, 1.3, 0.6, moe(3, 3, 10, 6))], 3, 2.0),
    # sizes of one: heads, channels, window, taps, experts, groups; no weight on a side
    "ones": conf(40, 61, [gla(left(1, 1, 2, 1, rot(1e4, 2), 1.0, 1), 1, 1, 1, 1.0, 1.0, 1.0, moe(1, 1, 8)),
                          ret(left(2, 2, 8, 8, rot(1e4, 4)), 2, 1, [0.75], rot(1e4, 2), 1.0, 0.0), delta(1, 1, 1, 2, 1, moe(2, 1, 1, 1))], 1, 0.5),
    # windows and sequences past a block and a chunk; many taps; heads that share keys
    "edge": conf(128, 80, [ret(left(8, 1, 32, 64, rot(3e5, 32), window=70), 64, 32, [0.95, 0.999], rot(1e6, 64), 1.0, 1.0, moe(8, 2, 64, 64)),
                           delta(6, 2, 32, 64, 7, moe(8, 1, 64, 64)),
                           gla(left(4, 4, 64, 32, rot(1e4, 32), cap=20.0), 4, 32, 64, 16.0, 0.8, 1.1)], 2, 3.0),
}


def settle_routing(w, js):
    """The choice of experts is a step function of its input: one direction of the stream per expert is
    the token's own, hardly touched by the sublayers, and the router reads those, so that rounding does not decide."""
    E = max([L["mlp"]["router"]["experts"] for L in js["layers"] if L["mlp"]] + [0])
    if E == 0:
        return
    assert E <= js["width"] // js["norm"]["groups"]
    g = torch.Generator().manual_seed(99)
    w["embed"][:, :E] = torch.stack([torch.randperm(E, generator=g).float() for _ in range(js["vocab"])]) * (6.0 / E) - 3.0
    for n, t in w.items():
        if n.endswith((".o", ".down")) and t.shape[0] == js["width"]:
            t[:E] *= 0.02
        elif n.endswith(("norm1", "norm2")):
            t[:E] = 1.0
        elif n.endswith("mlp.router"):
            t *= 0.02
            t[:, :E] += torch.eye(t.shape[0], E)


def make(name, device, dtype=F32, seed=0, tweak=None):
    js = CONFIGS[name] if isinstance(name, str) else name
    w = O.random_weights(js, seed)
    if dtype == BF16:
        settle_routing(w, js)
    if tweak:
        tweak(w)
    w = {k: v.to(BF16).float() for k, v in w.items()}
    return js, w, HybridModel(gezozen.config_from_json(js), device=device, dtype=dtype, weights=w)


def i32(device, *v):
    return torch.tensor(v, dtype=torch.int32, device=device)


def rnd(seed, *shape):
    return torch.randn(*shape, generator=torch.Generator().manual_seed(seed))


def slabs(x, S, seed, device, dtype):
    """x as a product of the dtype, or as S fp32 slabs that sum to it."""
    if S == 1:
        return x.to(device, dtype)
    part = rnd(seed, S - 1, *x.shape)
    return torch.cat([part, (x - part.sum(0))[None]]).to(device)


# ------------------------------------------------------------------ norms after the sum
def post_norm_case(device, dtype):
    for W, groups, rows, S, extra in ((30, 3, 3, 1, 0), (48, 48, 2, 2, 4), (64, 1, 5, 3, 8), (1024, 4, 2, 1, 64), (1280, 5, 2, 4, 0),
                                      (4096, 4, 3, 2, 128), (2050, 2, 1, 1, 1)):
        eps, alpha = 1e-3, 1.7
        x, y, z = rnd(1, rows, W), rnd(2, rows, W), rnd(3, rows, W)
        pre = rnd(4, rows, extra + W + 8)
        if S == 1:
            y, z, pre = (t.to(dtype).float() for t in (y, z, pre))
        b, w = rnd(5, W), rnd(6, W)
        eye = torch.eye(W)
        for q in (None, z):
            gate = torch.sigmoid(pre[:, extra:extra + W] + b) * (y if q is None else y + q)
            want = O.group_norm(alpha * x + gate, w, groups, eps)
            if W < 100 and q is None:      # the same through the oracle's own gate
                close(O.after_sum(pre[:, extra:extra + W], torch.zeros(rows, W), eye, b, alpha, w, groups, eps),
                      O.group_norm(alpha * pre[:, extra:extra + W], w, groups, eps))
            res = x.clone().to(device)
            out = ops.post_norm(slabs(y, S, 7, device, dtype), None if q is None else slabs(q, S, 8, device, dtype),
                                slabs(pre, S, 9, device, dtype), extra, b.to(device), res, alpha, w.to(device), groups, eps, dtype)
            assert out.dtype == dtype
            close(res, want, what=(W, groups))
            close(out, want, dtype, (W, groups))
        res = x.clone().to(device)
        close(ops.post_norm(None, None, None, 0, None, res, 1.0, w.to(device), groups, eps, dtype), O.group_norm(x, w, groups, eps), dtype)
    # parts of very different size: each has its own mean; eps decides in the small one
    x = torch.cat([rnd(1, 2, 24) * 1e3, rnd(2, 2, 24) * 1e-4, rnd(3, 2, 24)], 1)
    w = rnd(4, 72)
    res = x.clone().to(device)
    got = ops.post_norm(None, None, None, 0, None, res, 1.0, w.to(device), 3, 1e-3, F32).cpu()
    for k in range(3):
        close(got[:, 24 * k:24 * k + 24], O.group_norm(x, w, 3, 1e-3)[:, 24 * k:24 * k + 24])


# ------------------------------------------------------------------ rotation
def rope_case(device):
    for r in (rot(1e4, 2), rot(50.0, 16), rot(2e5, 64, (8.0, 1024.0, 32.0, 1.0)), rot(1e4, 32, (4.0, 64.0, 2.0, 2.0)), rot(300.0, 8, (16.0, 2e4, 50.0, 3.0)),
              rot(1e4, 16, (2.0, 3.0, 64.0, 1.0))):
        sc = r.get("scaling")
        R = Rotation(r["base"], r["dims"], sc and tuple(sc[k] for k in ("factor", "original", "fast", "slow")))
        f, m = R.frequencies()
        want, wm = O.frequencies(r)
        assert torch.allclose(f, torch.tensor(want, dtype=F64), rtol=1e-12) and abs(m - wm) < 1e-12
        pos = torch.tensor([0, 1, 7, 1000, 99999], dtype=torch.int32)
        cs = ops.rope_table(pos.to(device), f.to(device), m).cpu().double()
        a = pos.double()[:, None] * torch.tensor(want, dtype=F64)
        assert (cs - wm * torch.cat([a.cos(), a.sin()], -1)).abs().max() < 1e-6


# ------------------------------------------------------------------ attention
class Attend:
    """One sequence's attention through the operators, in portions, from a [q | k | v] projection."""

    def __init__(self, device, dtype, T, H, G, D, DV, r, bs, window=0, cap=0.0, bias=True, seed=0, rows=None, norms=None, scale=None):
        self.device, self.dtype, self.T, self.H, self.G, self.D, self.DV, self.bs = device, dtype, T, H, G, D, DV, bs
        self.window, self.cap, self.scale, self.eps = window, cap, scale or 1.5 * D ** -0.5, 1e-4
        n = (H + G) * D + G * DV
        self.rows = (rnd(seed, T, n) if rows is None else rows).to(dtype).float()
        self.bias = rnd(seed + 1, n) if bias else None
        self.qw, self.kw = (1 + 0.3 * rnd(seed + 2, D), 1 + 0.3 * rnd(seed + 3, D)) if norms is None else norms
        self.rot = rot(1e3, r, (4.0, 64.0, 8.0, 0.5) if seed % 2 else None)
        x = self.rows + (self.bias if bias else 0.0)
        q, k, v = x[:, :H * D].view(T, H, D), x[:, H * D:(H + G) * D].view(T, G, D), x[:, (H + G) * D:].view(T, G, DV)
        q, k = (O.rotate(O.rms(t, self.eps) * w, self.rot) for t, w in ((q, self.qw), (k, self.kw)))
        self.want = 0.8 * O.attend(q, k, v, self.scale, window, cap or None).reshape(T, -1)

    def run(self, cuts, S=1):
        dev, dt, bs, T = self.device, self.dtype, self.bs, self.T
        nb = (T + bs - 1) // bs
        perm = torch.randperm(nb + 3, generator=torch.Generator().manual_seed(T))[:nb].to(torch.int32)
        kc = torch.full((nb + 3, self.G, bs, self.D), 7.0, dtype=dt, device=dev)          # a former owner's rows
        vc = torch.full((nb + 3, self.G, bs, self.DV), 9.0, dtype=dt, device=dev)
        slots = torch.tensor([int(perm[t // bs]) * bs + t % bs for t in range(T)], dtype=torch.int32, device=dev)
        bt = perm[None].to(dev).contiguous()
        f, m = O.frequencies(self.rot)
        f = torch.tensor(f, dtype=F64, device=dev)
        up = lambda t: None if t is None else t.to(dev)  # noqa: E731
        W = self.H * self.DV
        out, t0 = [], 0
        for n in cuts:
            cs = ops.rope_table(torch.arange(t0, t0 + n, dtype=torch.int32, device=dev), f, m)
            x = torch.cat([self.rows[t0:t0 + n], torch.ones(n, 8)], 1)                 # other columns follow
            q = ops.qkv_rope_store(slabs(x, S, n, dev, dt), up(self.bias), up(self.qw), up(self.kw), cs, slots[t0:t0 + n], kc, vc,
                                   self.H, self.eps)
            wide = torch.full((n, W + 8), 5.0, dtype=dt, device=dev)
            kw = dict(window=self.window, v_cache=vc, cap=self.cap, out_scale=0.8, out=wide[:, :W])
            if n == 1 and t0 > 0:
                ops.window_attn(q, kc, bt, i32(dev, t0 + 1), self.scale, **kw)
            else:
                ops.window_attn(q, kc, bt, i32(dev, t0), self.scale, cu=i32(dev, 0, n), max_q=n, **kw)
            assert (wide[:, W:] == 5).all()
            out.append(wide[:, :W])
            t0 += n
        assert t0 == T
        return torch.cat(out)


ATTN_SIZES = ((23, 3, 3, 8, 8, 8, 16, 5, 0.0), (40, 4, 2, 16, 24, 8, 16, 1, 4.0), (75, 6, 2, 64, 32, 32, 64, 0, 8.0), (90, 8, 1, 32, 128, 16, 16, 33, 0.0),
              (140, 4, 4, 128, 64, 128, 64, 66, 0.0), (131, 6, 1, 96, 96, 24, 64, 0, 0.0), (70, 2, 1, 192, 200, 64, 32, 40, 2.0),
              (30, 3, 1, 10, 7, 6, 16, 9, 5.0), (20, 2, 2, 2, 1, 2, 16, 0, 0.0), (25, 2, 1, 264, 300, 10, 16, 12, 0.0))


def attention_case(device, dtype, sizes=ATTN_SIZES):
    for T, H, G, D, DV, r, bs, window, cap in sizes:
        A = Attend(device, dtype, T, H, G, D, DV, r, bs, window, cap, bias=T % 2 == 0, seed=T)
        for k, cuts in enumerate(([T], [2, 1, T - 3], [T - 6, 1, 1, 1, 1, 1, 1], [7, 1, 9, 2, T - 19])):
            close(A.run(cuts, S=1 + 2 * (k == 3)), A.want, dtype, (T, H, D, DV, cuts))


def window_edge_case(device, dtype):
    """One key outshines all others: a query sees it at distance window - 1 and not at distance
    window, in a prompt's portion and decoded; without a window, from any distance."""
    H, G, D, DV = 4, 2, 32, 16
    for window, j in ((8, 0), (8, 13), (64, 63), (65, 64), (70, 1), (129, 60), (0, 3)):
        T = j + (window or 150) + 3
        rows = rnd(window, T, (H + G) * D + G * DV) * 0.05
        q, k = rows[:, :H * D].view(T, H, D), rows[:, H * D:(H + G) * D].view(T, G, D)
        q[:, :, D - 1], k[:, :, D - 2] = 3.0, 1.0             # unrotated: every query looks along the last one,
        k[j, :, D - 2], k[j, :, D - 1] = 0.0, 1.0             # which only this key has
        rows[:, (H + G) * D:] *= 0.1
        rows[j, (H + G) * D:] = 5.0
        A = Attend(device, dtype, T, H, G, D, DV, 8, 16, window, 40.0 if window != 64 else 0.0, False, window, rows, (torch.ones(D), torch.ones(D)), 0.6)
        seen = A.want[:, 0]
        last = j + window - 1 if window else T - 1
        assert seen[last] > 3.5 and (not window or seen[j + window].abs() < 0.1)
        for cuts in ([T], [j + 1, *([1] * (T - j - 1))], [j + 1, (window or 60) - 2, 2, T - j - 1 - (window or 60)]):
            got = A.run([c for c in cuts if c > 0])
            close(got, A.want, dtype, (window, j, cuts))
            a = got.float().cpu()[:, 0]
            assert a[last] > 3.5 and (not window or a[j + window].abs() < 0.1), (window, j, cuts)


def soft_cap_case(device, dtype):
    """Scores far past the cap and far below it.  (What rounded queries and keys change in a score grows
    with the scale.)"""
    for scale, cap in ((40.0 if dtype == F32 else 6.0, 2.0), (0.01, 50.0), (3.0, 0.5)):
        A = Attend(device, dtype, 40, 2, 1, 32, 32, 16, 16, 0, cap, False, 4, scale=scale)
        for cuts in ([40], [38, 1, 1]):
            close(A.run(cuts), A.want, dtype, (scale, cap, cuts))


def batch_attention_case(device, dtype):
    """Packed sequences of unequal length and padded decode rows against each alone."""
    H, G, D, DV, bs = 6, 2, 24, 40, 16
    lens, ctx0 = [1, 33, 17, 2], [20, 0, 5, 40]
    g = torch.Generator().manual_seed(11)
    kc, vc = (torch.randn(24, G, bs, n, generator=g).to(device, dtype) for n in (D, DV))
    bt = torch.randperm(24, generator=g)[:20].view(4, 5).to(torch.int32).to(device)
    q = torch.randn(sum(lens), H * D, generator=g).to(device, dtype)
    cu = [0]
    for n in lens:
        cu.append(cu[-1] + n)
    kw = dict(window=28, v_cache=vc, cap=3.0)
    both = ops.window_attn(q, kc, bt, i32(device, *ctx0), 0.2, cu=i32(device, *cu), max_q=max(lens), **kw)
    for b, n in enumerate(lens):
        one = ops.window_attn(q[cu[b]:cu[b + 1]], kc, bt[b:b + 1].contiguous(), i32(device, ctx0[b]), 0.2, cu=i32(device, 0, n), max_q=n, **kw)
        close(both[cu[b]:cu[b + 1]], one.cpu(), dtype)
    dec = ops.window_attn(q[:4].contiguous(), kc, bt, i32(device, 21, 0, 80, 1), 0.2, **kw)
    assert torch.equal(dec[1].float().cpu(), torch.zeros(H * DV))           # a padded row
    for b, n in ((0, 21), (2, 80), (3, 1)):
        one = ops.window_attn(q[b:b + 1].contiguous(), kc, bt[b:b + 1].contiguous(), i32(device, n), 0.2, **kw)
        close(dec[b:b + 1], one.cpu(), dtype)


# ------------------------------------------------------------------ linear attention
class Linear:
    """One linear-attention recurrence over a sequence: rows [q | k | v | g | a | b] drawn at random,
    through the operators in portions, and by the oracle's recurrences."""

    def __init__(self, device, dtype, kind, T, H, G, d, vd, r=0, rank=5, seed=0, z_off=0.0, tau=4.0, decay=None):
        self.device, self.dtype, self.T, self.H, self.vd, self.kind, self.eps = device, dtype, T, H, vd, kind, 1e-4
        na, nb_ = {"channel": (rank, 0), "fixed": (0, 0), "delta": (H, H)}[kind]
        widths = [G * d, G * d, H * vd, H * vd, na, nb_]
        at = [8]
        for n in widths:
            at.append(at[-1] + n)
        self.rows = rnd(seed, T, at[-1] + 3).to(dtype).float()
        q, k, v, g, a, b = (self.rows[:, s:s + n] for s, n in zip(at, widths))
        self.norm = 1 + 0.3 * rnd(seed + 1, vd)
        self.b_gate, self.cs_rot, kw = None, None, {}
        qh, kh = q.reshape(T, G, d).double(), k.reshape(T, G, d).double()
        if kind == "channel":
            self.w_gate, self.b_gate = rnd(seed + 2, H * d, rank), rnd(seed + 3, H * d) + z_off
            al = O.sigmoid((a @ self.w_gate.T + self.b_gate).double()) ** (1 / tau)
            kw = dict(q_scale=d ** -0.5, inv_tau=1 / tau, rank=rank)
            o = O.linear_recurrence(qh * d ** -0.5, kh, v.reshape(T, H, vd).double(), al.view(T, H, d))
        elif kind == "fixed":
            dec = torch.tensor(decay or [0.9, 0.99, 0.999, 0.9999][:H], dtype=F64)
            self.w_gate, self.cs_rot = dec.log().float(), rot(1e3, r)
            qh, kh = O.rotate(qh, self.cs_rot), O.rotate(kh, self.cs_rot) * d ** -0.5
            kw = dict(k_scale=d ** -0.5)
            o = O.linear_recurrence(qh, kh, v.reshape(T, H, vd).double(), dec[None, :, None].expand(T, H, d))
        else:
            self.w_gate, self.b_gate = -torch.exp(rnd(seed + 2, H) - 1), rnd(seed + 3, H) + z_off
            qh, kh = (O.unit(x).repeat_interleave(H // G, 1) for x in (qh, kh))
            dec = torch.exp(self.w_gate.double() * O.softplus((a + self.b_gate).double()))
            kw = dict(q_scale=d ** -0.5)
            o = O.delta_recurrence(qh * d ** -0.5, kh, v.reshape(T, H, vd).double(), dec, O.sigmoid(b.double()))
        self.want = ((O.rms(o, self.eps) * self.norm).reshape(T, -1) * O.silu(g.double())).float()
        self.mix = ops.LinearMix(kind, H, G, d, vd, at[0], at[1], at[2], at[3], a=at[4], b=at[5], eps=self.eps, **kw)
        self.shape = ops.linear_state_shape(H, d, vd)

    def run(self, cuts, step=True, S=1):
        dev, dt = self.device, self.dtype
        up = lambda t: None if t is None else t.to(dev).contiguous()  # noqa: E731
        state = torch.zeros(3, *self.shape, device=dev)
        state[..., :self.vd] = 9.0                                         # a former owner's
        out, t0, W = [], 0, self.H * self.vd
        for n in cuts:
            X = slabs(self.rows[t0:t0 + n], S, n, dev, dt)
            cs = None
            if self.cs_rot is not None:
                f, m = O.frequencies(self.cs_rot)
                cs = ops.rope_table(torch.arange(t0, t0 + n, dtype=torch.int32, device=dev), torch.tensor(f, dtype=F64, device=dev), m)
            wide = torch.full((n, W + 4), 5.0, dtype=dt, device=dev)
            a = (X, X, self.mix, up(self.w_gate), up(self.b_gate), cs, up(self.norm), state, i32(dev, 1))
            if n == 1 and step:
                ops.linear_step(*a, i32(dev, t0), wide[:, 2:2 + W] if dt == F32 else wide[:, :W])
            else:
                ops.linear_scan(*a, i32(dev, 0, n), i32(dev, t0), n, wide[:, 2:2 + W] if dt == F32 else wide[:, :W])
            out.append(wide[:, 2:2 + W] if dt == F32 else wide[:, :W])
            assert int((wide == 5).sum()) >= 4 * n
            t0 += n
        assert t0 == self.T and (state[0, ..., :self.vd] == 9).all() and (state[2, ..., :self.vd] == 9).all()
        return torch.cat(out)


# kind, T, H, G, d, vd, rotated, rank
LINEAR_SIZES = (("channel", 70, 3, 3, 16, 24, 0, 5), ("channel", 131, 2, 2, 64, 40, 0, 16), ("channel", 150, 2, 2, 100, 130, 0, 3),
                ("channel", 40, 1, 1, 200, 33, 0, 7), ("channel", 9, 2, 2, 1, 1, 0, 1), ("channel", 66, 1, 1, 7, 300, 0, 300),
                ("fixed", 70, 3, 3, 16, 24, 12, 0), ("fixed", 140, 4, 4, 128, 64, 128, 0), ("fixed", 67, 2, 2, 9, 5, 2, 0), ("fixed", 45, 1, 1, 256, 16, 64, 0),
                ("delta", 70, 4, 2, 16, 24, 0, 0), ("delta", 140, 3, 1, 128, 128, 0, 0), ("delta", 129, 2, 2, 48, 72, 0, 0), ("delta", 67, 3, 3, 5, 7, 0, 0),
                ("delta", 50, 1, 1, 256, 20, 0, 0), ("delta", 20, 2, 1, 1, 1, 0, 0),
                # tall and wide states, whose step takes 16 waves or 4 lanes a row
                ("channel", 33, 1, 1, 160, 250, 0, 20), ("channel", 70, 1, 1, 128, 508, 0, 33), ("fixed", 33, 2, 2, 130, 100, 64, 0),
                ("delta", 66, 2, 1, 256, 256, 0, 0), ("fixed", 20, 1, 1, 64, 510, 8, 0))


def linear_case(device, dtype, sizes=LINEAR_SIZES):
    for kind, T, H, G, d, vd, r, rank in sizes:
        L = Linear(device, dtype, kind, T, H, G, d, vd, r, rank, seed=T + d)
        for k, cuts in enumerate(([T], [2] * (T // 2) + [1] * (T % 2), [1] * T, [T - 4, 1, 1, 2], [3, T - 5, 2])):
            close(L.run(cuts, S=1 + 2 * (k == 4)), L.want, dtype, (kind, T, H, d, vd, cuts[:4]))
        close(L.run([1, T - 2, 1], step=False), L.want, dtype, (kind, "scan of one token"))


def decay_case(device, dtype):
    """Decays near one over many chunks, and so strong that a chunk's product underflows; a constant decay of one."""
    for z_off, tau in ((-60.0, 0.25), (-8.0, 1.0), (30.0, 16.0)):
        L = Linear(device, dtype, "channel", 200, 2, 2, 24, 16, z_off=z_off, tau=tau, seed=3)
        for cuts in ([200], [70, 1, 129], [198, 1, 1]):
            close(L.run(cuts), L.want, dtype, (z_off, tau, cuts))
    for z_off in (-20.0, 60.0):
        L = Linear(device, dtype, "delta", 200, 2, 2, 24, 16, z_off=z_off, seed=4)
        for cuts in ([200], [70, 1, 129], [198, 1, 1]):
            close(L.run(cuts), L.want, dtype, ("delta", z_off, cuts))
    L = Linear(device, dtype, "fixed", 200, 3, 3, 24, 16, r=24, decay=[1.0, 1e-3, 0.9999], seed=5)
    for cuts in ([200], [70, 1, 129], [198, 1, 1]):
        close(L.run(cuts), L.want, dtype, ("fixed", cuts))


def batch_linear_case(device, dtype):
    """Packed sequences of unequal length -- empty ones among them --, new and carried, rows without a
    slot, against each alone."""
    for kind, G in (("channel", 3), ("fixed", 3), ("delta", 1)):
        L = Linear(device, dtype, kind, 210, 3, G, 16, 20, r=8, seed=9)
        lens, ctx0, sl = [1, 64, 0, 130, 2, 13], [7, 0, 0, 70, 3, 0], [4, 2, 0, -1, 1, 5]
        cu = [0]
        for n in lens:
            cu.append(cu[-1] + n)
        assert cu[-1] == 210
        up = lambda t: None if t is None else t.to(device).contiguous()  # noqa: E731
        st0 = torch.zeros(6, *L.shape)
        st0[..., :20] = rnd(10, 6, *L.shape[:2], 20)
        X = L.rows.to(device, dtype)
        cs = None
        if L.cs_rot is not None:
            pos = torch.cat([torch.arange(c, c + n) for c, n in zip(ctx0, lens)]).to(torch.int32)
            cs = ops.rope_table(pos.to(device), torch.tensor(O.frequencies(L.cs_rot)[0], dtype=F64, device=device))
        a = (L.mix, up(L.w_gate), up(L.b_gate))

        def scan(rows, cs_, state, slots, cu_, ctx, most):
            out = torch.empty(rows.shape[0], 60, dtype=dtype, device=device)
            return ops.linear_scan(rows, rows, *a, cs_, up(L.norm), state, i32(device, *slots), i32(device, *cu_), i32(device, *ctx), most, out)

        state = st0.clone().to(device)
        both = scan(X, cs, state, sl, cu, ctx0, max(lens))
        assert torch.equal(state[0].cpu(), st0[0]) and torch.equal(state[3].cpu(), st0[3])       # an empty sequence's, nobody's
        for b, n in enumerate(lens):
            if n == 0:
                continue
            s1, part = st0.clone().to(device), slice(cu[b], cu[b + 1])
            one = scan(X[part], cs[part] if cs is not None else None, s1, [sl[b]], [0, n], [ctx0[b]], n)
            close(both[part], one.cpu(), dtype, (kind, b))
            if sl[b] >= 0:
                close(state[sl[b]].reshape(3, -1), s1[sl[b]].cpu().reshape(3, -1), what=(kind, b))
        # one token a row, rows without a slot among them
        state, rows = st0.clone().to(device), X[:4].contiguous()
        out = torch.empty(4, 60, dtype=dtype, device=device)
        c4 = cs[:4].contiguous() if cs is not None else None
        ops.linear_step(rows, rows, *a, c4, up(L.norm), state, i32(device, 3, -1, 0, 5), i32(device, 9, 4, 0, 1), out)
        for b, (slot, pos) in enumerate(((3, 9), (-1, 4), (0, 0), (5, 1))):
            s1 = st0.clone().to(device)
            one = scan(rows[b:b + 1], c4[b:b + 1] if cs is not None else None, s1, [slot], [0, 1], [pos], 1)
            close(out[b:b + 1], one.cpu(), dtype, (kind, "step", b))
            if slot >= 0:
                close(state[slot].reshape(3, -1), s1[slot].cpu().reshape(3, -1), what=(kind, "step", b))
        assert torch.equal(state[1].cpu(), st0[1])


def forgotten_state_case(device, dtype):
    """A token's write is read back many chunks later through a decay of nearly one: a state lost between
    portions would leave nothing of it."""
    for kind in ("channel", "delta"):
        T, d, vd = 230, 32, 8
        L = Linear(device, dtype, kind, T, 1, 1, d, vd, rank=2, seed=6, z_off=40.0 if kind == "channel" else -40.0)
        at = L.mix
        L.rows[:, at.k:at.k + d] *= 0.01
        L.rows[:, at.q:at.q + d] = 0.0
        L.rows[:, at.q] = 2.0
        L.rows[:, at.k] = 0.0
        L.rows[5, at.k] = 8.0
        L.rows = L.rows.to(dtype).float()
        q, k, v, g = (L.rows[:, s:s + n].reshape(T, 1, -1).double() for s, n in ((at.q, d), (at.k, d), (at.v, vd), (at.g, vd)))
        if kind == "channel":
            z = L.rows[:, at.a:at.a + 2] @ L.w_gate.T + L.b_gate
            o = O.linear_recurrence(q * d ** -0.5, k, v, (O.sigmoid(z.double()) ** 0.25).view(T, 1, d))
        else:
            dec = torch.exp(L.w_gate.double() * O.softplus((L.rows[:, at.a:at.a + 1] + L.b_gate).double()))
            o = O.delta_recurrence(O.unit(q) * d ** -0.5, O.unit(k), v, dec, O.sigmoid(L.rows[:, at.b:at.b + 1].double()))
        assert o[-1].abs().max() > 0.05                       # still there
        L.want = ((O.rms(o, L.eps) * L.norm).reshape(T, -1) * O.silu(g.reshape(T, -1))).float()
        # (ahead of the write there is nothing to read but rounding)
        for cuts in ([T], [6, 64, 64, T - 134], [7] + [1] * (T - 7), [40, 2, 2, 1, T - 45]):
            close(L.run(cuts)[5:], L.want[5:], dtype, (kind, cuts[:4]))


def conv_case(device, dtype):
    """silu of the short convolution of the first columns of a wider projection, in portions, and in the
    step that hands the columns behind them on."""
    for C, NZ, taps, T in ((24, 8, 4, 40), (7, 5, 3, 9), (16, 40, 1, 12), (64, 12, 7, 35)):
        x = rnd(C, T, C + NZ + 4).to(dtype).float()
        w = rnd(C + 1, C, taps)
        want = O.short_conv(x[:, :C], w)
        wt = w.t().contiguous().to(device)
        for cuts in ([T], [2] * (T // 2) + [1] * (T % 2), [1] * T, [T - 3, 1, 2]):
            state, out, t0 = torch.full((3, taps - 1, C), 9.0, dtype=dtype, device=device), [], 0
            for n in cuts:
                p = x[t0:t0 + n].to(device, dtype)
                if n == 1:
                    y, z = ops.conv_step(p, wt, None, state, i32(device, 1), i32(device, t0), rest=NZ)
                    assert torch.equal(z.float().cpu(), x[t0:t0 + 1, C:C + NZ])
                else:
                    y = ops.causal_conv(p, wt, None, state, i32(device, 1), i32(device, 0, n), i32(device, t0), n)
                out.append(y)
                t0 += n
            close(torch.cat(out), want, dtype, (C, taps, cuts[:3]))
            assert (state[0] == 9).all() and (state[2] == 9).all()


# ------------------------------------------------------------------ experts
def expert_weights(E, F, W, K, seed):
    return rnd(seed, E, 2, F, K) * K ** -0.5, rnd(seed + 1, E, W, F) * F ** -0.5


MOE_SIZES = ((1, 64, 4, 1, 64, 0), (3, 64, 8, 2, 64, 32), (40, 96, 6, 3, 32, 64), (130, 128, 4, 2, 96, 0), (7, 36, 3, 3, 10, 6), (5, 40, 1, 1, 8, 0),
             (300, 128, 8, 2, 128, 64), (700, 192, 5, 1, 64, 0), (60, 64, 300, 4, 64, 0), (260, 64, 70, 16, 64, 64))


def moe_case(device, dtype, sizes=MOE_SIZES):
    """Routing, routed experts and the shared one, against the oracle."""
    for T, K, E, top, F, sh in sizes:
        x = rnd(T, T, K).to(dtype).float()
        wr = rnd(T + 1, E, K) * K ** -0.5
        # choices by rank of a few large elements: rounding does not decide
        g = torch.Generator().manual_seed(T)
        if E <= K // 2:
            x[:, :E] = torch.stack([torch.randperm(E, generator=g).float() for _ in range(T)]) / max(1, E) * 4 - 2
            wr[:, :E] += torch.eye(E) * 1.5
            wr[:, E:] *= 0.1
            wr[:, :E] -= wr[:, :E] * (1 - torch.eye(E)) * 0.9
        x, wr = x.to(dtype).float(), wr.to(dtype).float()
        up, down = (t.to(dtype).float() for t in expert_weights(E, F, K, K, T))
        t = {"router": wr}
        for e in range(E):
            t.update({f"e{e}.gate": up[e, 0], f"e{e}.up": up[e, 1], f"e{e}.down": down[e]})
        if sh:
            t.update({"shared.sg": rnd(3, 1, K).to(dtype).float() * 0.5, **{f"shared.{n}": (rnd(i, *s) * s[1] ** -0.5).to(dtype).float()
                      for i, (n, s) in enumerate((("gate", (sh, K)), ("up", (sh, K)), ("down", (K, sh))))}})
        m = {"router": {"experts": E, "top": top}, "shared": {"ff": sh} if sh else None}
        want = O.experts(x, m, t)
        w = torch.cat([wr] + ([t["shared.sg"]] if sh else [])).to(device, dtype)
        xd = x.to(device, dtype)
        ids, wts, rest = ops.moe_route(xd, w, E, top)
        s = O.sigmoid(x @ wr.T)
        best = torch.topk(s, top, -1)
        assert torch.equal(ids.cpu().sort(-1).values.long(), best.indices.sort(-1).values), (T, E, top)
        close(wts.sort(-1).values, best.values.sort(-1).values)
        y = ops.moe_experts(xd, ids, wts, up.to(device, dtype), down.to(device, dtype))
        assert y.shape == (top, T, K)
        y = y.float().sum(0)
        if sh:
            assert rest.shape == (T, 1)
            P = torch.cat([x, x @ t["shared.gate"].T, x @ t["shared.up"].T], 1)
            a = ops.glu(P.to(device), K, sh, rest, dtype)
            y = y + (a.float() @ t["shared.down"].T.to(device))
        close(y, want, dtype, (T, K, E, top, F, sh))


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
    assert got.dtype == F32


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


def long_case(name, device, dtype, T=150):
    """Long decoding, and a prompt of several chunks cut anywhere."""
    js, w, m = make(name, device, dtype, seed=6)
    seq = toks(T, js["vocab"], 10)
    want = O.forward(js, w, seq)
    for sizes in ([3] + [1] * (T - 3), [T], [64, 64], [63, 2, 66], [T - 20] + [1] * 20):
        close(run_steps(engine(m, bs=64), [[("a", p)] for p in portions(seq, sizes)])["a"], want, dtype, (name, sizes[:3]))


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
