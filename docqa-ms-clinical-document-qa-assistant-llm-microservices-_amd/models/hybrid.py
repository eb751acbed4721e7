"""Decoders made of attention, latent attention and recurrent (selective-scan, linear-attention)
mixers, with an fp32 residual stream.

A model is a list of layers (:class:`LayerSpec`: a mixer and an optional feed-forward) in one
of four forms: a norm before and after every sublayer, one after the other; with a
:class:`ParallelForm` one norm whose output both sublayers read, a convolution over time
ahead of the mixer and a second input from the token's side embedding; with a
:class:`PostNormForm` sublayers that read the stream itself, their gated results added to it and
the sum normed; with a :class:`PreNormForm` a norm before every sublayer alone, its result scaled
per channel ahead of the sum.  Layers may run
several passes over the same weights (``loop``), or use another layer's (``weights_of``).  Every
RUN of a layer has its own cache or
state, so the engine sees as many caches as runs; a latent-attention layer may read the cache
of an earlier one (``kv_from``) instead.

MI355X layout:
  * one sandwich_norm.hip launch stands between any two projections: it sums the split-K
    slabs of the last one, normalises that output, updates the fp32 residual (and adds the
    embedding ahead of a loop's next pass) and emits the next projection's input;
  * attention keeps the key rows as projected, once, as key and value, with the row's inverse
    RMS beside it (ops.qk_norm_store) -- half the cache bytes of a K / V pair;
  * a recurrent layer runs in_proj -> conv -> x_proj -> dt_proj -> scan + gate -> out_proj,
    conv and scan over packed sequences in prefill; in decode the conv step reads the in_proj
    slabs, and dt_proj, scan step and gate are one launch; the state is in per-request slots
    (engine/kv_cache.py StatePool);
  * the pre-norm form's stream update (slabs or the chosen experts' outputs summed and weighted,
    bias, layer scale) and the next norm are one launch;
  * latent attention caches one row a token for all heads and attends in one of two forms:
    with the key / value projections absorbed into the query and the output (decode, short
    portions: the cached row is key and value), or with keys and values of the visible rows
    made once by a GEMM (prompts); queries may come through a normed latent of their own, whose
    norm and the cache row are one launch; an output gate's rows are part of the input projection;
  * a linear-attention recurrence keeps one [key, value] matrix a head in fp32: decode is one launch
    from the projection's slabs to the gated heads, prompts run in chunks on fp32 MFMA; a mixer of
    two sides has one input projection, both sides write their part of one matrix, and one product
    projects it;
  * experts run as a grouped GEMM over (token, choice) rows sorted by expert (prompts), or one
    weight-streaming launch per projection that finds its rows itself (decode);
  * the post-norm form's gate rows are part of the sublayer's first projection, and one launch
    gates, adds, norms and updates the residual;
  * the parallel form's stream update, side input, next norm and (decode) convolution step are
    two launches around the side input's two small projections;
  * projections run on the same GEMM plans as the Llama decoder (ops.project / ops.linear):
    weights are padded with zero rows at load where that reaches a kernel's granule.

bf16 runs matrix products and activations in bf16; the residual, norms, attention scores,
decays, step sizes and states are fp32.  float32 runs everything in fp32.
"""
from __future__ import annotations

import math
import os
import zlib
from dataclasses import dataclass, field, replace

import torch

from .. import ops
from ..engine.kv_cache import KVSpec, StateSpec
from ..parallel import comm
from .decoder import Decoder
from .llama import AttnMeta


@dataclass(frozen=True)
class WindowAttentionSpec:
    """Causal attention over the last ``window`` tokens; no rotation; head-wise q / k norms;
    the key projection is the value; a learned sink per query head."""
    heads: int
    kv_heads: int
    dim: int
    scale: float
    window: int


@dataclass(frozen=True)
class SelectiveScanSpec:
    """Mamba mixer: ``inner`` channels, ``state`` states each, ``dt_rank`` of the step
    projection, ``conv`` taps of the short causal convolution."""
    inner: int
    state: int
    dt_rank: int
    conv: int


@dataclass(frozen=True)
class LatentAttentionSpec:
    """Causal attention over the last ``window`` tokens whose per-head keys (``dim``) and values
    (``vdim``) are linear in one normed latent of ``kv_rank`` a token, with ``rot_dim`` more
    query / key dimensions rotated by position (key part shared by the heads) and, unless ``sink``
    is off, a learned sink per head.  ``window`` 0: all tokens.  ``kv_from``: reads the latents of that
    layer's cache.  ``scaling``: as in :class:`Rotation`; ``interleaved``: rotated dimensions 2i and
    2i + 1 are a pair (else i and i + rot_dim / 2).  ``q_rank``: the queries are linear in a normed
    latent of their own.  ``gate``: the heads' outputs are multiplied by the sigmoid of a projection
    of the input, one number an "element" or one a "head"."""
    heads: int
    dim: int
    rot_dim: int
    vdim: int
    kv_rank: int
    scale: float
    window: int
    rope_base: float
    kv_from: int | None = None
    scaling: tuple | None = None
    interleaved: bool = False
    q_rank: int = 0
    gate: str = ""
    sink: bool = True

    @property
    def rot(self) -> Rotation:
        return Rotation(self.rope_base, self.rot_dim, self.scaling)


@dataclass(frozen=True)
class Rotation:
    """Rotary positions on a head's first ``dims`` dimensions, i paired with i + dims / 2.
    ``scaling``: YaRN's (factor, original, fast, slow) -- frequencies that turn fewer than ``slow``
    times in ``original`` tokens are divided by ``factor``, those beyond ``fast`` kept, a ramp
    between."""
    base: float
    dims: int
    scaling: tuple | None = None

    def frequencies(self) -> tuple:
        """(fp64 [dims / 2] angles per position, factor on cosines and sines)."""
        r = self.dims
        f = self.base ** (-torch.arange(0, r, 2, dtype=torch.float64) / r)
        if self.scaling is None:
            return f, 1.0
        factor, original, fast, slow = self.scaling

        def at(turns):
            return r * math.log(original / (2 * math.pi * turns)) / (2 * math.log(self.base))

        lo, hi = max(math.floor(at(fast)), 0), min(math.ceil(at(slow)), r - 1)
        ramp = ((torch.arange(r // 2, dtype=torch.float64) - lo) / max(hi - lo, 1e-3)).clamp(0, 1)
        return f / factor * ramp + f * (1 - ramp), 0.1 * math.log(factor) + 1


@dataclass(frozen=True)
class AttentionSpec:
    """Causal attention with normed, rotated queries and keys (over the last ``window`` tokens, 0:
    all), scores capped by ``softcap`` (0: not), biases on the projections where ``bias``."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    rot: Rotation
    window: int = 0
    softcap: float = 0.0
    bias: bool = False


@dataclass(frozen=True)
class GatedLinearSpec:
    """Gated linear attention: a decay sigmoid(z)^(1 / tau) per key channel, z a projection through
    ``rank`` elements (0: as the checkpoint's tensor has it)."""
    heads: int
    dim: int
    vdim: int
    tau: float
    rank: int = 0


@dataclass(frozen=True)
class RetentionSpec:
    """Linear attention with rotated queries and keys and a fixed decay per head."""
    heads: int
    dim: int
    vdim: int
    decay: tuple
    rot: Rotation


@dataclass(frozen=True)
class GatedDeltaSpec:
    """Gated delta rule: ``conv``-tap convolutions over q, k and v, unit q and k, the state's answer
    to the key subtracted from the value before it is written; ``heads`` share ``kv_heads`` q / k."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    conv: int


@dataclass(frozen=True)
class ChannelDeltaSpec:
    """Gated delta rule with a decay per head and key channel; the decay's logits and the output
    gate's (a sigmoid) are projections through ``a_rank`` and ``g_rank`` elements (0: as the
    checkpoint's tensors have it)."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    conv: int
    a_rank: int = 0
    g_rank: int = 0


@dataclass(frozen=True)
class TwoSidedSpec:
    """left_scale attention + right_scale linear attention of the same input."""
    left: AttentionSpec
    right: GatedLinearSpec | RetentionSpec
    left_scale: float
    right_scale: float


@dataclass(frozen=True)
class GroupRouter:
    """Softmax scores over the experts and ``identity`` more whose output is the input itself; chosen
    by score + a learned correction within the ``keep`` best of ``groups`` equal groups of
    neighbours; weights are the chosen scores over their sum, times ``scale``."""
    identity: int = 0
    groups: int = 1
    keep: int = 1
    scale: float = 1.0


@dataclass(frozen=True)
class MoESpec:
    """``top`` of ``experts`` SwiGLU feed-forwards of ``ff`` by sigmoid score, each reading the input
    times its score, and one of ``shared`` (0: none) for every token times a gate.  With a ``router``
    the outputs are weighted instead; ``limit`` > 0: gates clamped from above and up rows on both
    sides, g sigmoid(1.702 g) (u + 1)."""
    experts: int
    top: int
    ff: int
    shared: int = 0
    router: GroupRouter | None = None
    limit: float = 0.0


@dataclass(frozen=True)
class PreNormForm:
    """Layers x <- x + s1 * mixer(norm1(x)), x <- x + s2 * ff(norm2(x)), s1 and s2 a number per
    channel."""


@dataclass(frozen=True)
class PostNormForm:
    """Layers x <- norm(alpha x + sigmoid(W x + b) * sublayer(x)), the norm over ``groups`` equal
    parts of x."""
    alpha: float
    groups: int


@dataclass(frozen=True)
class ParallelForm:
    """Layers x <- x + mult (mixer(h + conv(h)) + ff(h)), h = norm1(x), then
    x <- x + mult rms(proj(gelu(gate x) * e)) * norm with e the layer's part of the token's
    side embedding.  ``conv`` taps, ``side`` elements of e."""
    mult: float
    conv: int
    side: int


@dataclass(frozen=True)
class LayerSpec:
    mixer: WindowAttentionSpec | SelectiveScanSpec | LatentAttentionSpec | TwoSidedSpec | GatedDeltaSpec | ChannelDeltaSpec
    ff: int = 0                     # feed-forward width, 0: none
    moe: MoESpec | None = None      # or experts (pre- and post-norm forms)
    weights_of: int | None = None   # the layer whose weights this one uses (pre-norm form)


@dataclass
class HybridConfig:
    name: str
    vocab_size: int
    hidden: int
    layer_specs: list
    embed_scale: float = 1.0
    rms_eps: float = 1e-5
    loop: tuple | None = None       # (start, stop, times)
    parallel: ParallelForm | None = None    # neither: norms around every sublayer
    post: PostNormForm | None = None
    pre: PreNormForm | None = None
    tied: bool = False              # the LM head is the embedding table
    act: str = ops.ACT_RELU2        # of the feed-forward
    norm_offset: float = 0.0        # added to the stored weights of the layers' and final norms
    logit_softcap: float | None = None
    max_position: int = 1 << 20     # no position enters the weights
    bos_token_id: int = -1          # no special tokens of its own
    eos_token_id: int = -1
    runs: list = field(init=False)  # (layer, embedding added ahead of it)

    def __post_init__(self):
        n = len(self.layer_specs)
        lo, hi, times = self.loop or (0, 0, 1)
        if not (0 <= lo <= hi <= n and times >= 1):
            raise ValueError(f"loop {self.loop} does not fit {n} layers")
        body = list(range(lo, hi))
        self.runs = [(i, False) for i in range(lo)]
        for p in range(times if body else 0):
            self.runs += [(i, p > 0 and i == lo) for i in body]
        self.runs += [(i, False) for i in range(hi, n)]
        if self.parallel is not None:
            if self.loop is not None or not all(isinstance(s.mixer, LatentAttentionSpec) for s in self.layer_specs):
                raise ValueError("parallel layers: latent attention, no loop")
            if self.parallel.conv < 1 or self.parallel.side < 1:
                raise ValueError(f"unsupported sizes {self.parallel}")
        if self.post is not None:
            if self.loop is not None or self.parallel is not None or self.hidden % self.post.groups:
                raise ValueError("post-norm layers: groups that divide the width, no loop")
        if self.pre is not None and (self.loop is not None or self.parallel is not None or self.post is not None):
            raise ValueError("pre-norm layers: no loop, no other form")
        if self.pre is not None and self.act != ops.ACT_POLY_NORM and any(sp.ff for sp in self.layer_specs):
            raise ValueError("pre-norm layers: dense feed-forwards with PolyNorm")
        for i, sp in enumerate(self.layer_specs):
            m = sp.mixer
            if (self.post is not None) != isinstance(m, (TwoSidedSpec, GatedDeltaSpec)) or (
                    sp.moe and self.post is None and self.pre is None) or (sp.ff and self.post is not None):
                raise ValueError("two-sided and delta mixers run in post-norm layers, experts in these or pre-norm ones")
            if self.post is not None:
                _check_post(sp)
            if (self.pre is not None) != isinstance(m, ChannelDeltaSpec) and not (
                    self.pre is not None and isinstance(m, LatentAttentionSpec)):
                raise ValueError("pre-norm layers: latent attention and channel-delta mixers")
            if self.pre is not None:
                _check_pre(sp, i, self.layer_specs)
            if isinstance(m, LatentAttentionSpec):
                if m.rot_dim % 2 or m.window < (0 if self.pre is not None else 1) or max(m.kv_rank, m.dim) > 2048 or min(
                        m.heads, m.dim, m.vdim, m.kv_rank, m.rot_dim) < 1:
                    raise ValueError(f"unsupported attention sizes {m}")
                if self.pre is None and (m.q_rank or m.gate or not m.sink):
                    raise ValueError("query latents and output gates run in pre-norm layers")
                if m.kv_from is not None:
                    src = self.layer_specs[m.kv_from].mixer if 0 <= m.kv_from < i else None
                    if not isinstance(src, LatentAttentionSpec) or src.kv_from is not None or (
                            (src.kv_rank, src.rot_dim, src.rope_base) != (m.kv_rank, m.rot_dim, m.rope_base)):
                        raise ValueError(f"layer {i}: kv_from {m.kv_from} is no earlier layer with such latents of its own")
                elif self.parallel is None and self.pre is None:
                    raise ValueError("latent attention runs in parallel and pre-norm layers")
            if isinstance(m, WindowAttentionSpec) and (m.heads % m.kv_heads or m.window < 1 or m.dim > 512):
                raise ValueError(f"unsupported attention sizes {m}")
            if isinstance(m, SelectiveScanSpec) and (m.state > 256 or m.conv < 1):
                raise ValueError(f"unsupported scan sizes {m}")

    @property
    def layers(self) -> int:
        return len(self.layer_specs)

    def tensor_shapes(self) -> dict:
        """Every weight's name and shape (linear weights [out, in])."""
        W, V = self.hidden, self.vocab_size
        out, par = {"embed": (V, W)}, self.parallel
        if self.post is not None:
            for i, sp in enumerate(self.layer_specs):
                out.update(_post_shapes(sp, W, f"l{i}."))
            out.update({"final.norm": (W,), "head": (V, W)})
            return out
        if self.pre is not None:
            for i, sp in enumerate(self.layer_specs):
                if sp.weights_of is None:
                    out.update(_pre_shapes(sp, W, f"l{i}."))
            out["final.norm"] = (W,)
            if not self.tied:
                out["head"] = (V, W)
            return out
        if par is not None:
            out["side.embed"] = (V, self.layers * par.side)
        for i, sp in enumerate(self.layer_specs):
            p, m = f"l{i}.", sp.mixer
            out[p + "norm1"] = (W,)
            if par is None:
                out[p + "norm1b"] = (W,)
            else:
                out.update({p + "canon1": (W, par.conv), p + "side.gate": (par.side, W), p + "side.proj": (W, par.side),
                            p + "side.norm": (W,)})
            if isinstance(m, LatentAttentionSpec):
                H, R = m.heads, m.kv_rank
                out.update({p + "mix.q": (H * (m.dim + m.rot_dim), W), p + "mix.uk": (H * m.dim, R),
                            p + "mix.uv": (H * m.vdim, R), p + "mix.sink": (H,), p + "mix.o": (W, H * m.vdim)})
                if m.kv_from is None:
                    out.update({p + "mix.dkv": (R + m.rot_dim, W), p + "mix.dkv.norm": (R,)})
            elif isinstance(m, WindowAttentionSpec):
                hd = m.heads * m.dim
                out.update({p + "mix.q": (hd, W), p + "mix.k": (m.kv_heads * m.dim, W), p + "mix.q.norm": (m.dim,),
                            p + "mix.k.norm": (m.dim,), p + "mix.sink": (m.heads,), p + "mix.o": (W, hd)})
            else:
                C, N, R = m.inner, m.state, m.dt_rank
                out.update({p + "mix.in": (2 * C, W), p + "mix.conv": (C, m.conv), p + "mix.conv.b": (C,),
                            p + "mix.x": (R + 2 * N, C), p + "mix.dt": (C, R), p + "mix.dt.b": (C,),
                            p + "mix.A_log": (C, N), p + "mix.D": (C,), p + "mix.o": (W, C)})
            if sp.ff:
                out.update({p + "mlp.up": (sp.ff, W), p + "mlp.down": (W, sp.ff)})
                if par is None:
                    out.update({p + "norm2": (W,), p + "norm2b": (W,)})
        out.update({"final.norm": (W,), "head": (V, W)})
        return out

    def num_params(self) -> int:
        """(a size that only the checkpoint knows counts as nothing)"""
        return sum(math.prod(s) for s in self.tensor_shapes().values())


def _check_state(s) -> None:
    if min(s.heads, s.dim, s.vdim) < 1 or s.heads % getattr(s, "kv_heads", 1):
        raise ValueError(f"unsupported sizes {s}")
    if s.dim > 256 or s.vdim > (512 if s.dim <= 128 else 256):
        raise ValueError(f"unsupported state sizes {s}")
    if getattr(s, "conv", 1) < 1:
        raise ValueError(f"unsupported sizes {s}")


def _check_pre(sp: LayerSpec, i: int, specs: list) -> None:
    m, f = sp.mixer, sp.moe
    if isinstance(m, ChannelDeltaSpec):
        _check_state(m)
    elif m.kv_from is not None or m.sink or m.gate not in ("", "head", "element") or not 0 <= m.q_rank <= 2048:
        raise ValueError(f"unsupported attention {m}")
    if f is not None:
        r = f.router
        if sp.ff or r is None or f.shared or f.limit <= 0:
            raise ValueError(f"pre-norm layers take clamped experts behind a group router, not {f}")
        n = f.experts + r.identity
        if not (1 <= f.experts and r.identity >= 0 and n <= 512 and f.ff >= 1 and 1 <= r.keep <= r.groups and n % r.groups == 0
                and 1 <= f.top <= min(16, r.keep * (n // r.groups))):
            raise ValueError(f"unsupported experts {f}")
    if sp.weights_of is not None:
        j = sp.weights_of
        if not 0 <= j < len(specs) or specs[j].weights_of is not None or replace(specs[j], weights_of=j) != sp:
            raise ValueError(f"layer {i}: weights_of {j} is no layer of the same kind with weights of its own")


def _check_post(sp: LayerSpec) -> None:
    m = sp.mixer
    sides = [m.left, m.right] if isinstance(m, TwoSidedSpec) else [m]
    for s in sides:
        if min(s.heads, s.dim, s.vdim) < 1 or s.heads % getattr(s, "kv_heads", 1):
            raise ValueError(f"unsupported sizes {s}")
        rot = getattr(s, "rot", None)
        if rot is not None and (rot.dims % 2 or not 2 <= rot.dims <= s.dim):
            raise ValueError(f"unsupported rotation {rot} of heads of {s.dim}")
        if isinstance(s, AttentionSpec):
            if s.dim > 512 or s.vdim > 512 or s.window < 0 or s.softcap < 0:
                raise ValueError(f"unsupported attention sizes {s}")
        else:
            _check_state(s)
        if isinstance(s, RetentionSpec) and (len(s.decay) != s.heads or not all(0 < d <= 1 for d in s.decay)):
            raise ValueError(f"one decay in (0, 1] per head expected: {s.decay}")
        if isinstance(s, GatedLinearSpec) and s.tau <= 0:
            raise ValueError(f"unsupported sizes {s}")
    if sp.moe is not None and not (1 <= sp.moe.top <= min(sp.moe.experts, 16) and sp.moe.ff >= 1 and sp.moe.shared >= 0
                                   and sp.moe.experts <= 512 and sp.moe.router is None and sp.moe.limit == 0):
        raise ValueError(f"unsupported experts {sp.moe}")


def _post_shapes(sp: LayerSpec, W: int, p: str) -> dict:
    out, m = {p + "norm1": (W,), p + "rg1": (W, W), p + "rg1.b": (W,)}, sp.mixer

    def linear(x, s):
        kv = getattr(s, "kv_heads", s.heads)
        out.update({x + "q": (kv * s.dim, W), x + "k": (kv * s.dim, W), x + "v": (s.heads * s.vdim, W),
                    x + "g": (s.heads * s.vdim, W), x + "o": (W, s.heads * s.vdim)})

    if isinstance(m, GatedDeltaSpec):
        x = p + "mix."
        linear(x, m)
        out.update({x + "q.conv": (m.kv_heads * m.dim, m.conv), x + "k.conv": (m.kv_heads * m.dim, m.conv),
                    x + "v.conv": (m.heads * m.vdim, m.conv), x + "b": (m.heads, W), x + "a": (m.heads, W),
                    x + "A_log": (m.heads,), x + "dt_bias": (m.heads,), x + "norm": (m.vdim,)})
    else:
        x, s = p + "mix.left.", m.left
        sizes = {"q": s.heads * s.dim, "k": s.kv_heads * s.dim, "v": s.kv_heads * s.vdim}
        out.update({x + n: (r, W) for n, r in sizes.items()})
        if s.bias:
            out.update({f"{x}{n}.b": (r,) for n, r in sizes.items()})
        out.update({x + "q.norm": (s.dim,), x + "k.norm": (s.dim,), x + "o": (W, s.heads * s.vdim)})
        x, s = p + "mix.right.", m.right
        linear(x, s)
        if isinstance(s, GatedLinearSpec):
            n = s.heads * s.dim
            out.update({x + "norm": (s.vdim,), x + "a1": (s.rank, W), x + "a2": (n, s.rank), x + "a2.b": (n,)})
    if sp.moe is not None:
        x, f = p + "mlp.", sp.moe
        out.update({p + "norm2": (W,), p + "rg2": (W, W), p + "rg2.b": (W,), x + "router": (f.experts, W)})
        sizes = {f"e{e}.": f.ff for e in range(f.experts)}
        if f.shared:
            sizes["shared."] = f.shared
            out[x + "shared.sg"] = (1, W)
        for n, ff in sizes.items():
            out.update({x + n + "gate": (ff, W), x + n + "up": (ff, W), x + n + "down": (W, ff)})
    return out


def _pre_shapes(sp: LayerSpec, W: int, p: str) -> dict:
    x, m, f = p + "mix.", sp.mixer, sp.moe
    out = {p + "norm1": (W,), p + "ls1": (W,), x + "o": (W, m.heads * m.vdim)}
    if isinstance(m, ChannelDeltaSpec):
        key, val, a, g = m.kv_heads * m.dim, m.heads * m.vdim, m.a_rank, m.g_rank
        out.update({x + "q": (key, W), x + "q.conv": (key, m.conv), x + "k": (key, W), x + "k.conv": (key, m.conv),
                    x + "v": (val, W), x + "v.conv": (val, m.conv), x + "b": (m.heads, W), x + "A_log": (m.heads,),
                    x + "norm": (m.vdim,), x + "a1": (a, W), x + "a2": (m.heads * m.dim, a), x + "dt_bias": (m.heads * m.dim,),
                    x + "g1": (g, W), x + "g2": (val, g)})
    else:
        q = m.heads * (m.dim + m.rot_dim)
        out.update({x + "dq": (m.q_rank, W), x + "dq.norm": (m.q_rank,), x + "uq": (q, m.q_rank)} if m.q_rank else {x + "q": (q, W)})
        out.update({x + "dkv": (m.kv_rank + m.rot_dim, W), x + "dkv.norm": (m.kv_rank,), x + "uk": (m.heads * m.dim, m.kv_rank),
                    x + "uv": (m.heads * m.vdim, m.kv_rank)})
        if m.gate:
            out[x + "g"] = (m.heads * (m.vdim if m.gate == "element" else 1), W)
    if sp.ff or f is not None:
        out.update({p + "norm2": (W,), p + "ls2": (W,)})
    x = p + "mlp."
    if sp.ff:
        out.update({x + "up": (sp.ff, W), x + "up.b": (sp.ff,), x + "down": (W, sp.ff), x + "down.b": (W,), x + "act": (4,)})
    elif f is not None:
        n = f.experts + f.router.identity
        out.update({x + "router": (n, W), x + "correction": (n,)})
        for e in range(f.experts):
            out.update({f"{x}e{e}.gate": (f.ff, W), f"{x}e{e}.up": (f.ff, W), f"{x}e{e}.down": (W, f.ff)})
    return out


# Feed-forward weights from which a captured decode step runs a parallel layer's sublayers as two
# branches of the graph: 352 MB (width 4096, ff 21504) 1.07 -> 0.98 ms a step of 8 layers at batch 1,
# 1.92 -> 1.69 at 64, 2.52 -> 2.47 at 256; 100 MB lose 6 % at batch 1 to 16
FORK_MIN_BYTES = int(os.environ.get("DOCQA_FORK_MIN_MB", "192")) << 20


def _pad_up(n: int, m: int) -> int:
    return -(-n // m) * m


@dataclass
class _Part:
    """Rows [lo, hi) of a forward that attend / scan together: one token a row (decode) or
    packed sequences (prefill)."""
    lo: int
    hi: int
    meta: AttnMeta

    @property
    def decode(self) -> bool:
        return not self.meta.prefill


class _Keys:
    """The visible keys of a prompt batch under one window (0: all): every sequence's [first, end) rows,
    packed (``cu``), and how many there are."""

    def __init__(self, spans: list, window: int, device):
        lo = [max(0, a - window + 1) if window else 0 for a, _ in spans]
        cu = [0]
        for k, (_, e) in zip(lo, spans):
            cu.append(cu[-1] + e - k)
        t = torch.tensor(lo + cu, dtype=torch.int32)
        t = (t.pin_memory() if device.type == "cuda" else t).to(device, non_blocking=True)
        self.first, self.cu, self.total = t[:len(lo)], t[len(lo):], cu[-1]
        self.tokens = sum(e - a for a, e in spans)

        def seen(n):           # (query, key) pairs of positions below n
            k = min(n, window) if window else n
            return k * (k + 1) // 2 + (n - k) * window

        self.pairs = sum(seen(e) - seen(a) for a, e in spans)


@dataclass
class _Forward:
    """What the layers of one forward share: tables by :class:`Rotation`, the visible keys of
    prompts by window."""
    rope: dict
    keys: dict


def _split(t: torch.Tensor, part: _Part, parts: list) -> torch.Tensor:
    return t if len(parts) == 1 else t[part.lo:part.hi]


def _join(ts: list) -> torch.Tensor:
    return ts[0] if len(ts) == 1 else torch.cat(ts)


class WindowAttention:
    def __init__(self, sp: WindowAttentionSpec, get, eps: float, dtype):
        self.sp, self.eps = sp, eps
        self.qk = torch.cat([get("q"), get("k")]).to(dtype).contiguous()
        self.o = get("o").to(dtype).contiguous()
        # the cached key is the projection itself: both norm weights go to the query side
        self.qk_norm = (get("q.norm").float() * get("k.norm").float()).contiguous()
        self.sink = get("sink").float().contiguous()

    def cache_spec(self):
        return KVSpec(self.sp.kv_heads, self.sp.dim, shared=True)

    def activation_elems(self) -> int:
        return (3 * self.sp.heads + self.sp.kv_heads) * self.sp.dim

    def run(self, x, parts, slot_mapping, cache, decode):
        sp = self.sp
        kc, ks = cache
        q = ops.qk_norm_store(ops.project(x, self.qk, decode), self.qk_norm, slot_mapping, kc, ks, sp.heads, self.eps)
        out = []
        for p in parts:
            m = p.meta
            kw = dict(window=sp.window, sink=self.sink, k_scale=ks)
            if p.decode:
                out.append(ops.window_attn(_split(q, p, parts), kc, m.block_tables, m.context_lens, sp.scale, **kw))
            else:
                out.append(ops.window_attn(_split(q, p, parts), kc, m.block_tables, m.prefix_lens, sp.scale,
                                           cu=m.cu_seqlens, max_q=m.max_len, **kw))
        return ops.project(_join(out), self.o, decode)


class SelectiveScan:
    def __init__(self, sp: SelectiveScanSpec, get, eps: float, dtype):
        self.sp, self.dtype = sp, dtype
        C, N, R = sp.inner, sp.state, sp.dt_rank
        self.w_in = get("in").to(dtype).contiguous()
        self.conv_w = get("conv").float().t().contiguous()        # [taps, C]
        self.conv_b = get("conv.b").float().contiguous()
        # [dt | B | C] rows, each section and the whole padded with zero rows to the GEMM granules
        self.rp, self.np = _pad_up(R, 64), _pad_up(N, 8)
        wx = get("x")
        rows = self.rp + 2 * self.np
        pad = wx.new_zeros(_pad_up(rows, 128 if rows <= 256 else 256), C)
        pad[:R] = wx[:R]
        pad[self.rp:self.rp + N] = wx[R:R + N]
        pad[self.rp + self.np:self.rp + self.np + N] = wx[R + N:]
        self.w_x = pad.to(dtype).contiguous()
        wd = get("dt")
        self.w_dt = torch.cat([wd, wd.new_zeros(C, self.rp - R)], 1).to(dtype).contiguous()
        self.dt_b = get("dt.b").float().contiguous()
        a = -torch.exp(get("A_log").float()) * math.log2(math.e)
        self.A2 = torch.cat([a, a.new_zeros(C, _pad_up(N, 4) - N)], 1).contiguous()
        self.D = get("D").float().contiguous()
        self.w_o = get("o").to(dtype).contiguous()

    def cache_spec(self):
        return StateSpec(((self.sp.conv - 1, self.sp.inner), tuple(self.A2.shape)), (False, True))

    def activation_elems(self) -> int:
        return 5 * self.sp.inner + self.w_x.shape[0]

    def run(self, x, parts, slot_mapping, cache, decode):
        C, N = self.sp.inner, self.sp.state
        conv_state, scan_state = cache
        xz = ops.project(x, self.w_in, True) if decode and len(parts) == 1 else ops.linear(x, self.w_in, decode)
        xc, zs = [], []
        for p in parts:
            m = p.meta
            if p.decode:
                y, z = ops.conv_step(_split(xz, p, parts), self.conv_w, self.conv_b, conv_state, m.state_slots,
                                     m.positions)
            else:
                r = _split(xz, p, parts)
                y, z = ops.causal_conv(r, self.conv_w, self.conv_b, conv_state, m.state_slots, m.cu_seqlens,
                                       m.prefix_lens, m.max_len), r[:, C:]
            xc.append(y)
            zs.append(z)
        xa = _join(xc)
        dt_in, bc = ops.slab_columns(ops.project(xa, self.w_x, decode), self.rp, 2 * self.np, self.dtype)
        out = []
        for p, y, z in zip(parts, xc, zs):
            m = p.meta
            r = _split(dt_in, p, parts)
            args = (_split(bc, p, parts), 0, self.np, N, z, self.A2, self.D, self.dt_b, scan_state, m.state_slots)
            if p.decode:       # the step projection runs inside the step
                out.append(ops.selective_step(y, (r, self.w_dt), *args, m.positions))
            else:
                out.append(ops.selective_scan(y, ops.linear(r, self.w_dt), *args, m.cu_seqlens, m.prefix_lens, m.max_len))
        return ops.project(_join(out), self.w_o, decode)


class LatentAttention:
    def __init__(self, sp: LatentAttentionSpec, get, eps: float, dtype):
        self.sp, self.eps, self.dtype = sp, eps, dtype
        H, d, vd, R = sp.heads, sp.dim, sp.vdim, sp.kv_rank
        self.d8, self.r8, self.R8, self.v8 = (_pad_up(n, 8) for n in (d, sp.rot_dim, R, vd))
        self.rot = sp.rot
        # the kernels pair rotated dimension i with i + rot_dim / 2: neighbours become that by the order
        # of the projections' rows, the same one for queries and keys
        order = torch.arange(sp.rot_dim)
        if sp.interleaved:
            order = torch.cat([order[0::2], order[1::2]])

        def paired(t, keep):           # rows [.., keep | rotated]
            t = t.view(-1, keep + sp.rot_dim, t.shape[-1])
            return torch.cat([t[:, :keep], t[:, keep:][:, order.to(t.device)]], 1).flatten(0, 1)

        # q (or its latent) | latent | key part | gate
        rows = [get("dq") if sp.q_rank else paired(get("q"), d)] + ([paired(get("dkv"), R)] if sp.kv_from is None else [])
        self.q_norm = self.w_uq = self.gate_at = None
        if sp.q_rank:
            self.q_norm = get("dq.norm").float().contiguous()
            self.w_uq = _joint([paired(get("uq"), d)], dtype)
        if sp.gate:
            n = sum(t.shape[0] for t in rows)
            self.gate_at = _pad_up(n, 8)
            rows += [rows[0].new_zeros(self.gate_at - n, rows[0].shape[1]), get("g")]
        self.w_in = _joint(rows, dtype)
        self.c_norm = get("dkv.norm").float().contiguous() if sp.kv_from is None else None
        uk, uv = get("uk").view(H, d, R), get("uv").view(H, vd, R)
        pad = torch.nn.functional.pad
        # absorbed: query heads into the latent space, attended latents to values
        self.w_qc = pad(uk.transpose(1, 2), (0, self.d8 - d, 0, self.R8 - R)).to(dtype).contiguous()   # [H, R8, d8]
        self.w_cv = pad(uv, (0, self.R8 - R)).to(dtype).contiguous()                                   # [H, vd, R8]
        # expanded: every head's keys, then values
        self.w_kv = None
        if ops.packed_attn_ok(dtype, self.d8, self.r8, vd):
            kv = torch.cat([pad(uk, (0, self.R8 - R, 0, self.d8 - d)).reshape(H * self.d8, self.R8),
                            pad(uv, (0, self.R8 - R, 0, self.v8 - vd)).reshape(H * self.v8, self.R8)])
            n = kv.shape[0]
            self.w_kv = pad(kv, (0, 0, 0, _pad_up(n, 256 if n >= 1024 else 64) - n)).to(dtype).contiguous()
        self.sink = get("sink").float().contiguous() if sp.sink else None
        self.o = get("o").to(dtype).contiguous()

    def cache_spec(self):
        """Its own rows, or (``kv_from``) the index of the run whose rows it reads."""
        return KVSpec(1, self.R8 + self.r8, latent=True) if self.sp.kv_from is None else self.sp.kv_from

    def activation_elems(self) -> int:
        H = self.sp.heads
        return (self.w_in.shape[0] + H * (self.d8 + self.r8 + self.sp.vdim) + 2 * H * (self.d8 + self.v8)
                + (self.w_uq.shape[0] + self.sp.q_rank if self.sp.q_rank else 0))

    def _expanded(self, keys: _Keys | None) -> bool:
        """Whether making keys and values of the visible rows costs less than attending in the
        latent space (multiply-adds a head; the absorbed projections are one product a query)."""
        if keys is None or self.w_kv is None:
            return False
        kv = self.d8 + self.v8
        return (keys.total * self.R8 * kv + keys.pairs * (kv + self.r8)
                < keys.tokens * self.R8 * kv + keys.pairs * (2 * self.R8 + self.r8))

    def run(self, x, parts, slot_mapping, cache, decode, fw: _Forward):
        sp, cs = self.sp, fw.rope[self.rot]
        P = Q = ops.project(x, self.w_in, decode)
        c_norm = self.c_norm
        if sp.q_rank:
            cq = ops.latent_norm_store(P, cs, slot_mapping, cache, self.q_norm, c_norm, self.eps, self.dtype)
            Q, c_norm = ops.project(cq, self.w_uq, decode), None
        q = ops.latent_store(Q, cs, slot_mapping, cache, c_norm, sp.heads, sp.dim, sp.kv_rank, self.eps, self.dtype)
        out = []
        for p in parts:
            m, qp = p.meta, _split(q, p, parts)
            keys = None if p.decode else fw.keys.get(sp.window)
            kw = dict(window=sp.window, sink=self.sink,
                      gate=(P, self.gate_at, sp.vdim if sp.gate == "head" else 1, p.lo) if sp.gate else None)
            if self._expanded(keys):
                c, kr = ops.latent_gather(cache, m.block_tables, keys.first, keys.cu, keys.total, self.R8)
                out.append(ops.packed_window_attn(qp, ops.linear(c, self.w_kv), kr, sp.heads, sp.dim, sp.vdim, m.cu_seqlens,
                                                  keys.cu, m.max_len, sp.scale, **kw))
                continue
            qc = ops.head_project(qp, self.w_qc, self.r8)
            if p.decode:
                a = ops.latent_attn(qc, cache, m.block_tables, m.context_lens, sp.scale, self.w_cv, **kw)
            else:
                a = ops.latent_attn(qc, cache, m.block_tables, m.prefix_lens, sp.scale, self.w_cv, cu=m.cu_seqlens,
                                    max_q=m.max_len, **kw)
            out.append(a)
        return ops.project(_join(out), self.o, decode)


class MLP:
    """down(act(up x))."""

    def __init__(self, get, dtype, act: str):
        self.up = get("up").to(dtype).contiguous()
        self.down = get("down").to(dtype).contiguous()
        self.act = act
        self.nbytes = 2 * self.up.numel() * self.up.element_size()

    def run(self, x, decode):
        return ops.project(ops.act_linear(x, self.up, self.act, decode), self.down, decode)


class PolyNormMLP:
    """down(act(up x + b)) with act the four-term PolyNorm; its own bias goes to the stream update."""

    def __init__(self, get, dtype, eps: float):
        up, down = get("up"), get("down")
        self.n, self.eps, self.dtype = up.shape[0], eps, dtype
        pad = _pad_up(self.n, 64) - self.n
        self.up = _joint([up], dtype)
        self.up_b, self.act = get("up.b").float().contiguous(), get("act").float().contiguous()
        self.down = torch.nn.functional.pad(down, (0, pad)).to(dtype).contiguous()
        self.down_b = get("down.b").float().contiguous()

    def activation_elems(self) -> int:
        return self.up.shape[0] + self.down.shape[1]

    def run(self, x, decode):
        a = ops.poly_norm(ops.project(x, self.up, decode), self.up_b, self.act, self.down.shape[1], self.eps, self.dtype)
        return ops.project(a, self.down, decode), {"bias": self.down_b}


def _joint(rows: list, dtype) -> torch.Tensor:
    """One weight of several projections of the same input, padded with zero rows to the GEMM granules."""
    n = sum(t.shape[0] for t in rows)
    pad = rows[0].new_zeros(_pad_up(n, 256 if n >= 1024 else 64) - n, rows[0].shape[1])
    return torch.cat([*rows, pad]).to(dtype).contiguous()


def _in_project(x, w, parts: list, decode: bool):
    """A projection whose consumers take slabs, if one part has all of its rows, else the product."""
    return ops.project(x, w, decode) if len(parts) == 1 else ops.linear(x, w, decode)


class Attention:
    """The attention side of a mixer: rows [q | k | v] of its input projection."""

    def __init__(self, sp: AttentionSpec, get, eps: float, dtype, out_scale: float):
        self.sp, self.eps, self.out_scale = sp, eps, out_scale
        self.rows = [get(n) for n in "qkv"]
        self.n = sum(t.shape[0] for t in self.rows)
        self.bias = torch.cat([get(n + ".b") for n in "qkv"]).float().contiguous() if sp.bias else None
        self.q_norm, self.k_norm = (get(n + ".norm").float().contiguous() for n in "qk")
        self.o = get("o")

    def cache_spec(self):
        return KVSpec(self.sp.kv_heads, self.sp.dim, v_dim=self.sp.vdim)

    def run(self, P, parts, slot_mapping, cache, fw, out):
        sp = self.sp
        kc, vc = cache
        q = ops.qkv_rope_store(P, self.bias, self.q_norm, self.k_norm, fw.rope[sp.rot], slot_mapping, kc, vc, sp.heads, self.eps)
        for p in parts:
            m = p.meta
            kw = dict(window=sp.window, v_cache=vc, cap=sp.softcap, out_scale=self.out_scale, out=_split(out, p, parts))
            if p.decode:
                ops.window_attn(_split(q, p, parts), kc, m.block_tables, m.context_lens, sp.scale, **kw)
            else:
                ops.window_attn(_split(q, p, parts), kc, m.block_tables, m.prefix_lens, sp.scale, cu=m.cu_seqlens,
                                max_q=m.max_len, **kw)


class LinearAttention:
    """A linear-attention recurrence: rows [q | k | v | g | a | b] of its input projection, from
    column ``at`` on."""

    def __init__(self, sp, get, eps: float, dtype, at: int = 0, out_scale: float = 1.0):
        self.sp, self.rot = sp, None
        kv = getattr(sp, "kv_heads", sp.heads)
        names, kw, self.b_gate = ["q", "k", "v", "g"], {}, None
        norm = torch.ones(sp.vdim, device=get("o").device)
        if isinstance(sp, GatedLinearSpec):
            kind, norm = "channel", get("norm").float()
            names.append("a1")
            self.w_gate, self.b_gate = get("a2").float().contiguous(), get("a2.b").float().contiguous()
            kw = dict(q_scale=sp.dim ** -0.5, inv_tau=1.0 / sp.tau, rank=self.w_gate.shape[1])
        elif isinstance(sp, ChannelDeltaSpec):
            # decays, gates and steps come as one matrix of their own (ops.low_rank)
            kind, norm, names = "channel_delta", get("norm").float(), ["q", "k", "v"]
            self.w_gate, self.b_gate = (-torch.exp(get("A_log").float())).contiguous(), get("dt_bias").float().contiguous()
            kw = dict(q_scale=sp.dim ** -0.5, gate="sigmoid")
        elif isinstance(sp, RetentionSpec):
            kind, self.rot = "fixed", sp.rot
            self.w_gate = torch.tensor(sp.decay, dtype=torch.float64).log().float().to(norm.device)
            kw = dict(k_scale=sp.dim ** -0.5)
        else:
            kind, norm = "delta", get("norm").float()
            names += ["a", "b"]
            self.w_gate, self.b_gate = (-torch.exp(get("A_log").float())).contiguous(), get("dt_bias").float().contiguous()
            kw = dict(q_scale=sp.dim ** -0.5)
        self.norm = (norm * out_scale).contiguous()
        self.rows = [get(n) for n in names]
        cols = [at]
        for t in self.rows:
            cols.append(cols[-1] + t.shape[0])
        self.n = cols[-1] - at
        if kind == "channel_delta":
            n = sp.heads * sp.dim
            cols = cols[:3] + [n, 0, n + sp.heads * sp.vdim]
        self.mix = ops.LinearMix(kind, sp.heads, kv, sp.dim, sp.vdim, *cols[:4], a=cols[4], b=cols[5] if kind.endswith("delta") else 0,
                                 eps=eps, **kw)
        self.o = get("o")

    def state_shape(self) -> tuple:
        return ops.linear_state_shape(self.sp.heads, self.sp.dim, self.sp.vdim)

    def cache_spec(self):
        return StateSpec((self.state_shape(),), (True,))

    def run_part(self, X, Z, mix, p: _Part, state, cs, out):
        m = p.meta
        a = (X, Z, mix, self.w_gate, self.b_gate, cs, self.norm, state, m.state_slots)
        if p.decode:
            ops.linear_step(*a, m.positions, out)
        else:
            ops.linear_scan(*a, m.cu_seqlens, m.prefix_lens, m.max_len, out)

    def run(self, P, parts, state, fw, out):
        for p in parts:
            x = _split(P, p, parts)
            cs = _split(fw.rope[self.rot], p, parts) if self.rot is not None else None
            self.run_part(x, x, self.mix, p, state[0], cs, _split(out, p, parts))


class TwoSidedMixer:
    """Attention and linear attention of the same input, scaled and added: one input projection of
    both sides (and the ``tail`` rows), one product of both results."""

    def __init__(self, sp: TwoSidedSpec, get, eps: float, dtype, tail):
        self.left = Attention(sp.left, lambda n: get("left." + n), eps, dtype, sp.left_scale)
        self.right = LinearAttention(sp.right, lambda n: get("right." + n), eps, dtype, self.left.n, sp.right_scale)
        self.tail = self.left.n + self.right.n
        self.w_in = _joint(self.left.rows + self.right.rows + [tail], dtype)
        self.split = self.left.o.shape[1]
        self.o = torch.cat([self.left.o, self.right.o], 1).to(dtype).contiguous()
        self.left.rows = self.right.rows = self.left.o = self.right.o = None

    def rotations(self) -> set:
        return {r for r in (self.left.sp.rot, self.right.rot) if r is not None}

    def cache_specs(self) -> list:
        return [self.left.cache_spec(), self.right.cache_spec()]

    def activation_elems(self) -> int:
        lf, r = self.left.sp, self.right.sp
        return self.w_in.shape[0] + 2 * self.o.shape[1] + lf.heads * lf.dim + 2 * r.heads * (4 * r.dim + 2 * r.vdim + 64)

    def run(self, x, parts, slot_mapping, cache, decode, fw: _Forward):
        P = _in_project(x, self.w_in, parts, decode)
        out = x.new_empty(x.shape[0], self.o.shape[1])
        self.left.run(P, parts, slot_mapping, cache[0], fw, out[:, :self.split])
        self.right.run(P, parts, cache[1], fw, out[:, self.split:])
        return ops.project(out, self.o, decode), P, self.tail


class DeltaMixer:
    """Gated delta rule behind short convolutions of q, k and v."""

    def __init__(self, sp: GatedDeltaSpec, get, eps: float, dtype, tail):
        self.sp = sp
        self.lin = LinearAttention(sp, get, eps, dtype)
        self.conv_w = torch.cat([get(n + ".conv") for n in "qkv"]).float().t().contiguous()      # [taps, C]
        self.C = self.conv_w.shape[1]
        self.tail = self.lin.n
        self.rest = self.tail - self.C                     # gate, decay and step columns
        m = self.lin.mix
        self.step_mix = replace(m, g=m.g - self.C, a=m.a - self.C, b=m.b - self.C)
        self.w_in = _joint(self.lin.rows + [tail], dtype)
        self.o = self.lin.o.to(dtype).contiguous()
        self.lin.rows = self.lin.o = None

    def rotations(self) -> set:
        return set()

    def cache_specs(self) -> list:
        return [StateSpec(((self.sp.conv - 1, self.C), self.lin.state_shape()), (False, True))]

    def activation_elems(self) -> int:
        sp = self.sp
        return self.w_in.shape[0] + self.C + self.o.shape[1] + 2 * sp.heads * (4 * sp.dim + 3 * sp.vdim + 64)

    def run(self, x, parts, slot_mapping, cache, decode, fw: _Forward):
        conv_state, state = cache[0]
        one = decode and len(parts) == 1
        P = ops.project(x, self.w_in, True) if one else ops.linear(x, self.w_in, decode)
        out = x.new_empty(x.shape[0], self.o.shape[1])
        for p in parts:
            m, r = p.meta, _split(P, p, parts)
            if p.decode:
                y, z = ops.conv_step(r, self.conv_w, None, conv_state, m.state_slots, m.positions, rest=self.rest)
                mix = self.step_mix
            else:
                y, z = ops.causal_conv(r, self.conv_w, None, conv_state, m.state_slots, m.cu_seqlens, m.prefix_lens, m.max_len), r
                mix = self.lin.mix
            self.lin.run_part(y, z, mix, p, state, None, _split(out, p, parts))
        return ops.project(out, self.o, decode), P, self.tail


class ChannelDelta:
    """Gated delta rule with channel decays behind short convolutions of q, k and v.  One projection
    [q k v | decay's and gate's inner elements | steps]; a second product makes decays and gates of theirs."""

    def __init__(self, sp: ChannelDeltaSpec, get, eps: float, dtype):
        self.sp = sp
        pad = torch.nn.functional.pad
        self.lin = LinearAttention(sp, get, eps, dtype)
        self.conv_w = torch.cat([get(n + ".conv") for n in "qkv"]).float().t().contiguous()      # [taps, C]
        self.C = self.conv_w.shape[1]
        inner = [pad(t, (0, 0, 0, _pad_up(t.shape[0], 8) - t.shape[0])) for t in (get("a1"), get("g1"))]
        self.ranks = tuple(t.shape[0] for t in inner)
        self.rest = sum(self.ranks) + sp.heads
        self.w_a, self.w_g = (pad(t, (0, k - t.shape[1])).to(dtype).contiguous() for t, k in zip((get("a2"), get("g2")), self.ranks))
        self.w_in = _joint([*self.lin.rows, *inner, get("b")], dtype)
        self.o = self.lin.o.to(dtype).contiguous()
        self.lin.rows = self.lin.o = None

    def cache_spec(self):
        return StateSpec(((self.sp.conv - 1, self.C), self.lin.state_shape()), (False, True))

    def activation_elems(self) -> int:
        sp = self.sp
        return self.w_in.shape[0] + self.C + self.o.shape[1] + 2 * sp.heads * (6 * sp.dim + 5 * sp.vdim + 64)

    def run(self, x, parts, slot_mapping, cache, decode, fw: _Forward):
        conv_state, state = cache
        one = decode and len(parts) == 1
        P = ops.project(x, self.w_in, True) if one else ops.linear(x, self.w_in, decode)
        out = x.new_empty(x.shape[0], self.o.shape[1])
        for p in parts:
            m, r = p.meta, _split(P, p, parts)
            if p.decode:
                y, z = ops.conv_step(r, self.conv_w, None, conv_state, m.state_slots, m.positions, rest=self.rest)
                at = 0
            else:
                y, z = ops.causal_conv(r, self.conv_w, None, conv_state, m.state_slots, m.cu_seqlens, m.prefix_lens, m.max_len), r
                at = self.C
            self.lin.run_part(y, ops.low_rank(z, at, self.w_a, self.w_g, self.sp.heads), self.lin.mix, p, state, None,
                              _split(out, p, parts))
        return ops.project(out, self.o, decode)


def _expert_weights(sp: MoESpec, get, dtype) -> tuple:
    """([E, 2 (gate, up), F, W], [E, W, F]), F padded with zeros to 64."""
    pad = torch.nn.functional.pad
    F = _pad_up(sp.ff, 64)
    up = torch.stack([torch.stack([pad(get(f"e{e}.{n}").to(dtype), (0, 0, 0, F - sp.ff)) for n in ("gate", "up")])
                      for e in range(sp.experts)])
    return up, torch.stack([pad(get(f"e{e}.down").to(dtype), (0, F - sp.ff)) for e in range(sp.experts)])


class GroupExperts:
    """Experts behind a group router, identity experts among them; the stream update weighs and sums
    the chosen ones' outputs."""

    def __init__(self, sp: MoESpec, get, dtype):
        self.sp = sp
        self.up, self.down = _expert_weights(sp, get, dtype)
        self.router, self.correction = get("router").to(dtype).contiguous(), get("correction").float().contiguous()

    def activation_elems(self) -> int:
        return self.sp.top * (self.up.shape[2] + self.up.shape[3])

    def run(self, x, decode):
        sp, r = self.sp, self.sp.router
        ids, wts = ops.moe_route_groups(x, self.router, self.correction, sp.top, r.groups, r.keep, r.scale)
        return ops.moe_experts(x, ids, wts, self.up, self.down, sp.limit), {"mix": (ids, wts, sp.experts, x)}


class Experts:
    """Routed experts and a shared one.  The shared expert's gate and up rows and the ``tail`` rows
    are one projection; routing is fp32."""

    def __init__(self, sp: MoESpec, get, dtype, tail):
        self.sp, self.dtype = sp, dtype
        pad = torch.nn.functional.pad
        self.up, self.down = _expert_weights(sp, get, dtype)
        router, rows = [get("router")], [tail]
        self.shared = None
        if sp.shared:
            self.fs = _pad_up(sp.shared, 64)
            rows = [pad(get("shared." + n), (0, 0, 0, self.fs - sp.shared)) for n in ("gate", "up")] + rows
            self.shared = pad(get("shared.down").to(dtype), (0, self.fs - sp.shared)).contiguous()
            router.append(get("shared.sg"))
        self.router = torch.cat(router).to(dtype).contiguous()
        self.tail = 2 * self.fs if sp.shared else 0
        self.w_in = _joint(rows, dtype)

    def activation_elems(self) -> int:
        return self.w_in.shape[0] + self.sp.top * (self.up.shape[2] + self.up.shape[3]) + self.tail

    def run(self, x, decode):
        P = ops.project(x, self.w_in, decode)
        ids, wts, sg = ops.moe_route(x, self.router, self.sp.experts, self.sp.top)
        y = ops.moe_experts(x, ids, wts, self.up, self.down)
        if self.shared is None:
            return y, None, P, self.tail
        return y, ops.project(ops.glu(P, 0, self.fs, sg, self.dtype), self.shared, decode), P, self.tail


class InputConv:
    """h + conv(h): the causal convolution per channel ahead of a mixer, the identity in its
    last tap."""

    def __init__(self, w):
        self.w = w.float().t().clone(memory_format=torch.contiguous_format)      # [taps, W]
        self.w[-1] += 1.0

    def cache_spec(self):
        return StateSpec((((self.w.shape[0] - 1), self.w.shape[1]),), (False,))

    def run(self, h, parts, state):
        out = []
        for p in parts:
            m, x = p.meta, _split(h, p, parts)
            if p.decode:
                out.append(ops.conv_step(x, self.w, None, state, m.state_slots, m.positions, silu=False)[0])
            else:
                out.append(ops.causal_conv(x, self.w, None, state, m.state_slots, m.cu_seqlens, m.prefix_lens, m.max_len,
                                           silu=False))
        return _join(out)


class SideInput:
    """proj(gelu(gate x) * e), e = columns [col, col + n) of the token's side embedding."""

    def __init__(self, get, dtype, col: int):
        gate, proj = get("gate"), get("proj")
        n = gate.shape[0]
        pad = _pad_up(n, 256 if n > 128 else 64) - n                # zero rows: a zero gate
        self.gate = torch.cat([gate, gate.new_zeros(pad, gate.shape[1])]).to(dtype).contiguous()
        self.proj = torch.cat([proj, proj.new_zeros(proj.shape[0], pad)], 1).to(dtype).contiguous()
        self.col, self.n = col, n

    def run(self, x, ids, table, decode):
        return ops.side_project(ops.narrow_project(x, self.gate, decode), ids, table, self.col, self.n, self.proj, decode)


class HybridModel(Decoder):
    prefix_reuse = False      # a prompt's recurrent state is not in its K/V blocks
    paged_prefill = True

    def __init__(self, cfg: HybridConfig, device="cuda", dtype=torch.bfloat16, seed: int = 0, weights=None):
        """``weights``: mapping of :meth:`HybridConfig.tensor_shapes` names to tensors, read one
        at a time; None: random ones."""
        if comm.state().tp_size > 1:
            raise NotImplementedError("hybrid decoders run at TP = 1 (replicate them per GPU)")
        self.cfg, self.device, self.dtype = cfg, torch.device(device), dtype
        self.tp, self.tp_rank = 1, 0
        self.vocab_shard = self.vocab_valid = cfg.vocab_size
        self.vocab_start = 0
        att = [getattr(s.mixer, "left", s.mixer) for s in cfg.layer_specs if not isinstance(s.mixer, SelectiveScanSpec)]
        self.hq, self.hkv = (att[0].heads, getattr(att[0], "kv_heads", 1)) if att else (1, 1)
        self._side_stream = None  # second branch of captured decode steps
        self.tap = None           # a list: receives the residual stream after every run
        self._load(weights if weights is not None else _RandomWeights(cfg, self.device, seed))

    def _load(self, weights) -> None:
        cfg, dt = self.cfg, self.dtype
        shapes = cfg.tensor_shapes()

        def get(name):
            t = weights[name]
            if len(t.shape) != len(shapes[name]) or any(n not in (0, k) for n, k in zip(shapes[name], t.shape)):
                raise ValueError(f"{name}: shape {tuple(t.shape)}, expected {shapes[name]}")
            return t.to(self.device)

        def vec(name):
            return get(name).float().contiguous()

        def norm(name):
            return vec(name) + cfg.norm_offset if cfg.norm_offset else vec(name)

        par = cfg.parallel
        self.embed = get("embed").to(dt).contiguous()
        self.lm_head = self.embed if cfg.tied else get("head").to(dt).contiguous()
        self.final_norm = norm("final.norm")
        self.layers, self.rope_freq, self.windows = [], {}, []
        if cfg.pre is not None:
            own = {}
            for i, sp in enumerate(cfg.layer_specs):
                if sp.weights_of is not None:
                    continue
                p = f"l{i}."
                L = own[i] = {"mixer": _MIXERS[type(sp.mixer)](sp.mixer, lambda n: get(p + "mix." + n), cfg.rms_eps, dt),
                              "norm1": norm(p + "norm1"), "ls1": vec(p + "ls1"), "mlp": None}
                if sp.ff or sp.moe is not None:
                    tensor = lambda n: get(p + "mlp." + n)  # noqa: E731
                    L.update(mlp=PolyNormMLP(tensor, dt, cfg.rms_eps) if sp.ff else GroupExperts(sp.moe, tensor, dt),
                             norm2=norm(p + "norm2"), ls2=vec(p + "ls2"))
            self.layers = [own[i if sp.weights_of is None else sp.weights_of] for i, sp in enumerate(cfg.layer_specs)]
            self._load_rotations()
            return
        if cfg.post is not None:
            for i, sp in enumerate(cfg.layer_specs):
                p = f"l{i}."
                L = {"mixer": _MIXERS[type(sp.mixer)](sp.mixer, lambda n: get(p + "mix." + n), cfg.rms_eps, dt, get(p + "rg1")),
                     "norm1": norm(p + "norm1"), "rg1_b": vec(p + "rg1.b"), "mlp": None}
                if sp.moe is not None:
                    L.update(mlp=Experts(sp.moe, lambda n: get(p + "mlp." + n), dt, get(p + "rg2")), norm2=norm(p + "norm2"),
                             rg2_b=vec(p + "rg2.b"))
                self.layers.append(L)
            for rot in {r for L in self.layers for r in L["mixer"].rotations()}:
                f, mult = rot.frequencies()
                self.rope_freq[rot] = (f.to(self.device), mult)
            return
        for i, sp in enumerate(cfg.layer_specs):
            p = f"l{i}."
            L = {"mixer": _MIXERS[type(sp.mixer)](sp.mixer, lambda n: get(p + "mix." + n), cfg.rms_eps, dt),
                 "norm1": norm(p + "norm1"), "mlp": None}
            if sp.ff:
                L["mlp"] = MLP(lambda n: get(p + "mlp." + n), dt, cfg.act)
            if par is not None:
                L.update(conv=InputConv(get(p + "canon1")), side_norm=vec(p + "side.norm") * par.mult,
                         side=SideInput(lambda n: get(p + "side." + n), dt, i * par.side))
            else:
                L["norm1b"] = norm(p + "norm1b")
                if sp.ff:
                    L.update(norm2=norm(p + "norm2"), norm2b=norm(p + "norm2b"))
            self.layers.append(L)
        if par is not None:
            self.side_embed = get("side.embed").to(dt).contiguous()
            self._load_rotations()

    def _load_rotations(self) -> None:
        """Of the latent-attention layers: the rotations, and the windows whose keys prompts expand."""
        latent = [L["mixer"] for L in self.layers if isinstance(L["mixer"], LatentAttention)]
        for rot in {m.rot for m in latent}:
            f, mult = rot.frequencies()
            self.rope_freq[rot] = (f.to(self.device), mult)
        self.windows = sorted({m.sp.window for m in latent if m.w_kv is not None})

    # ------------------------------------------------------------------ caches
    def _run_specs(self) -> list:
        """Per run: what its mixer keeps (or, an integer, whose cache it reads), what its input
        convolution keeps."""
        if self.cfg.post is not None:
            return [L["mixer"].cache_specs() for L in self.layers]
        return [[self.layers[i][k].cache_spec() for k in ("mixer", "conv") if k in self.layers[i]]
                for i, _ in self.cfg.runs]

    def kv_specs(self) -> list:
        return [s for run in self._run_specs() for s in run if isinstance(s, KVSpec)]

    def state_specs(self) -> list:
        return [s for run in self._run_specs() for s in run if isinstance(s, StateSpec)]

    def bind_caches(self, kv, state) -> list:
        """Per run its mixer's tensors (the pre-norm form's latent rows as one); in the parallel form (latent rows, convolution inputs), in the
        post-norm form a tuple of tensors for each of its mixer's specs."""
        k, s = iter(kv.caches), iter(state.states if state is not None else [])
        out = []
        for run in self._run_specs():
            own = [next(k) if isinstance(sp, KVSpec) else next(s) if isinstance(sp, StateSpec) else out[sp] for sp in run]
            if self.cfg.post is not None:
                out.append(own)
                continue
            if self.cfg.pre is not None:
                out.append(own[0][0] if isinstance(run[0], KVSpec) else own[0])
                continue
            out.append(own[0] if len(own) == 1 else (own[0][0], own[1][0]))
        return out

    def activation_elems(self) -> int:
        if self.cfg.post is not None or self.cfg.pre is not None:
            return 10 * self.cfg.hidden + max([max(L["mixer"].activation_elems(), L["mlp"].activation_elems() if L["mlp"] else 0)
                                               for L in self.layers] + [0])
        ff = max([s.ff for s in self.cfg.layer_specs] + [0])
        return 8 * self.cfg.hidden + max(max(L["mixer"].activation_elems() for L in self.layers), 3 * ff)

    def weight_bytes(self) -> int:
        return self.cfg.num_params() * self.embed.element_size()

    # ------------------------------------------------------------------ forward
    def forward(self, input_ids, meta: AttnMeta, caches: list, logits_index=None, greedy_ids: bool = False):
        """Same arguments and result as :meth:`LlamaModel.forward`; prefill metadata always carries block
        tables, prefix lengths and state slots."""
        x = self._hidden(input_ids, [_Part(0, input_ids.shape[0], meta)], meta.slot_mapping, caches)
        return self._head(x, logits_index, greedy_ids)

    def forward_mixed(self, input_ids, n_dec: int, dmeta: AttnMeta, pmeta: AttnMeta, caches: list, logits_index,
                      return_logits: bool = False):
        """Same arguments and result as :meth:`LlamaModel.forward_mixed`: rows [0, n_dec) decode, the rest
        prompt portions; projections run over all rows at once."""
        T = input_ids.shape[0]
        parts = ([_Part(0, n_dec, dmeta)] if n_dec else []) + ([_Part(n_dec, T, pmeta)] if T > n_dec else [])
        slots = _join([p.meta.slot_mapping for p in parts])
        return self._head(self._hidden(input_ids, parts, slots, caches), logits_index, not return_logits)

    def _hidden(self, input_ids, parts, slot_mapping, caches):
        if self.cfg.parallel is not None:
            return self._hidden_parallel(input_ids, parts, slot_mapping, caches)
        if self.cfg.post is not None:
            return self._hidden_post(input_ids, parts, slot_mapping, caches)
        if self.cfg.pre is not None:
            return self._hidden_pre(input_ids, parts, slot_mapping, caches)
        cfg, eps, dt = self.cfg, self.cfg.rms_eps, self.dtype
        decode = all(p.decode for p in parts)
        runs = cfg.runs
        loops = any(again for _, again in runs)
        first = self.layers[runs[0][0]]["norm1"] if runs else self.final_norm
        res, emb, x = ops.embed_scale_rmsnorm(input_ids, self.embed, cfg.embed_scale, first, eps, keep=loops)
        for r, (i, _) in enumerate(runs):
            L = self.layers[i]
            last = r + 1 == len(runs)
            nxt = self.final_norm if last else self.layers[runs[r + 1][0]]["norm1"]
            add = emb if not last and runs[r + 1][1] else None
            y = L["mixer"].run(x, parts, slot_mapping, caches[r], decode)
            if L["mlp"] is not None:
                x = ops.sandwich_rmsnorm(y, res, L["norm1b"], L["norm2"], eps, out_dtype=dt)
                y = L["mlp"].run(x, decode)
            x = ops.sandwich_rmsnorm(y, res, L["norm1b" if L["mlp"] is None else "norm2b"], nxt, eps, add=add,
                                     out_dtype=dt)
            if self.tap is not None:
                self.tap.append(res - add if add is not None else res.clone())
        return x

    def _shared(self, parts) -> _Forward:
        pos = _join([p.meta.positions for p in parts])
        fw = _Forward({r: ops.rope_table(pos, f, mult) for r, (f, mult) in self.rope_freq.items()}, {})
        for p in parts:
            if not p.decode and p.meta.spans is not None:
                fw.keys = {w: _Keys(p.meta.spans, w, self.device) for w in self.windows}
        return fw

    def _hidden_pre(self, input_ids, parts, slot_mapping, caches):
        cfg, eps, dt = self.cfg, self.cfg.rms_eps, self.dtype
        decode = all(p.decode for p in parts)
        fw = self._shared(parts)
        norms = [L["norm1"] for L in self.layers] + [self.final_norm]
        res, _, x = ops.embed_scale_rmsnorm(input_ids, self.embed, cfg.embed_scale, norms[0], eps)
        for L, cache, nxt in zip(self.layers, caches, norms[1:]):
            y = L["mixer"].run(x, parts, slot_mapping, cache, decode, fw)
            x = ops.scaled_rmsnorm(y, res, L["ls1"], nxt if L["mlp"] is None else L["norm2"], eps, out_dtype=dt)
            if L["mlp"] is not None:
                y, kw = L["mlp"].run(x, decode)
                x = ops.scaled_rmsnorm(y, res, L["ls2"], nxt, eps, out_dtype=dt, **kw)
            if self.tap is not None:
                self.tap.append(res.clone())
        return x

    def _hidden_parallel(self, input_ids, parts, slot_mapping, caches):
        cfg, eps, dt = self.cfg, self.cfg.rms_eps, self.dtype
        decode = all(p.decode for p in parts)
        fw = self._shared(parts)
        first = self.layers[0]["norm1"] if self.layers else self.final_norm
        res, _, h = ops.embed_scale_rmsnorm(input_ids, self.embed, cfg.embed_scale, first, eps)
        hm = self.layers[0]["conv"].run(h, parts, caches[0][1]) if self.layers else h
        for i, L in enumerate(self.layers):
            y, f = self._sublayers(L, h, hm, parts, slot_mapping, caches[i][0], decode, fw)
            xs = ops.add_scaled(y, f, res, cfg.parallel.mult, dt)
            y = L["side"].run(xs, input_ids, self.side_embed, decode)
            if i + 1 == len(self.layers):
                h = ops.sandwich_rmsnorm(y, res, L["side_norm"], self.final_norm, eps, out_dtype=dt)
            else:
                nxt, state = self.layers[i + 1], caches[i + 1][1]
                if decode:
                    m = parts[0].meta
                    h, hm = ops.sandwich_rmsnorm_conv(y, res, L["side_norm"], nxt["norm1"], eps, nxt["conv"].w, state,
                                                      m.state_slots, m.positions)
                else:
                    h = ops.sandwich_rmsnorm(y, res, L["side_norm"], nxt["norm1"], eps, out_dtype=dt)
                    hm = nxt["conv"].run(h, parts, state)
            if self.tap is not None:
                self.tap.append(res.clone())
        return h

    def _hidden_post(self, input_ids, parts, slot_mapping, caches):
        cfg, eps, dt = self.cfg, self.cfg.rms_eps, self.dtype
        alpha, groups = cfg.post.alpha, cfg.post.groups
        decode = all(p.decode for p in parts)
        fw = self._shared(parts)
        res, _, x = ops.embed_scale_rmsnorm(input_ids, self.embed, cfg.embed_scale, None, eps)
        for L, cache in zip(self.layers, caches):
            y, P, col = L["mixer"].run(x, parts, slot_mapping, cache, decode, fw)
            x = ops.post_norm(y, None, P, col, L["rg1_b"], res, alpha, L["norm1"], groups, eps, dt)
            if L["mlp"] is not None:
                y, z, P, col = L["mlp"].run(x, decode)
                x = ops.post_norm(y, z, P, col, L["rg2_b"], res, alpha, L["norm2"], groups, eps, dt)
            if self.tap is not None:
                self.tap.append(res.clone())
        return ops.post_norm(None, None, None, 0, None, res, 1.0, self.final_norm, groups, eps, dt)

    def _sublayers(self, L, h, hm, parts, slot_mapping, cache, decode, fw):
        """The layer's mixer and feed-forward (or None).  In a captured decode step they are two
        branches of the graph: the mixer's chain of small launches runs beside the feed-forward's
        two weight-streaming ones."""
        if L["mlp"] is None:
            return L["mixer"].run(hm, parts, slot_mapping, cache, decode, fw), None
        fork = (decode and h.is_cuda and L["mlp"].nbytes >= FORK_MIN_BYTES and torch.cuda.is_current_stream_capturing())
        if not fork:
            return L["mixer"].run(hm, parts, slot_mapping, cache, decode, fw), L["mlp"].run(h, decode)
        if self._side_stream is None:
            self._side_stream = torch.cuda.Stream(self.device)
        main = torch.cuda.current_stream()
        # h outlives the join below and f is consumed after it, so neither is handed out again while
        # the other stream may still use it
        self._side_stream.wait_stream(main)
        with torch.cuda.stream(self._side_stream):
            f = L["mlp"].run(h, decode)
        y = L["mixer"].run(hm, parts, slot_mapping, cache, decode, fw)
        main.wait_stream(self._side_stream)
        return y, f

    def _head(self, x, logits_index, greedy_ids):
        if logits_index is not None:
            x = x.index_select(0, logits_index)
        if greedy_ids:
            return self.greedy_ids(x)          # (a soft cap keeps the order of the logits)
        logits = ops.lm_head_logits(x.contiguous(), self.lm_head)
        return logits if self.cfg.logit_softcap is None else ops.soft_cap(logits, self.cfg.logit_softcap)


_MIXERS = {WindowAttentionSpec: WindowAttention, SelectiveScanSpec: SelectiveScan, LatentAttentionSpec: LatentAttention,
           TwoSidedSpec: TwoSidedMixer, GatedDeltaSpec: DeltaMixer, ChannelDeltaSpec: ChannelDelta}


class _RandomWeights:
    """Random weights by tensor name: unit-variance projections, a decay spectrum and step
    sizes in the range of trained selective-scan models."""

    def __init__(self, cfg: HybridConfig, device, seed: int):
        self.shapes, self.device, self.seed, self.offset = cfg.tensor_shapes(), device, seed, cfg.norm_offset

    def __getitem__(self, name: str) -> torch.Tensor:
        shape = self.shapes[name]
        g = torch.Generator(device=self.device)
        g.manual_seed((self.seed * 1_000_003 + zlib.crc32(name.encode())) & 0x7FFFFFFFFFFF)
        kind = name.rsplit(".", 1)[-1]
        if name.endswith("norm") or kind.startswith("norm"):
            stored_off = self.offset if kind.startswith(("norm1", "norm2")) or name == "final.norm" else 0.0
            return torch.full(shape, 1.0 - stored_off, device=self.device)
        if kind in ("ls1", "ls2", "act"):
            return torch.full(shape, 1.0 if kind != "act" else 1 / 3, device=self.device)
        if kind == "correction":
            return torch.zeros(shape, device=self.device)
        if kind == "A_log" and len(shape) == 1:
            return torch.empty(shape, device=self.device).uniform_(1.0, 16.0, generator=g).log()
        if kind == "A_log":
            return torch.log(torch.arange(1, shape[1] + 1, device=self.device).float()).expand(shape).contiguous()
        if kind == "D":
            return torch.ones(shape, device=self.device)
        if name.endswith(("dt.b", "dt_bias")):
            u = torch.rand(shape, device=self.device, generator=g)
            dt = torch.exp(u * (math.log(0.1) - math.log(1e-3)) + math.log(1e-3))
            return dt + torch.log(-torch.expm1(-dt))          # softplus^-1
        std = 1.0 if len(shape) == 1 else (0.02 if name == "embed" else shape[-1] ** -0.5)
        t = torch.empty(shape, device=self.device, dtype=torch.bfloat16 if len(shape) == 2 else torch.float32)
        return t.normal_(0.0, std, generator=g)
