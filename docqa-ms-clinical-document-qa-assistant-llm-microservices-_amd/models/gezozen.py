"""The Gezozen decoder: its config.json, tensor names and presets, on models/hybrid.py.

config.json: ``architecture`` "Gezozen", ``vocab``, ``width``, ``postln_alpha``, ``norm`` (``eps``,
``groups``) and ``layers``: ``type`` "parallel" (attention beside gated linear attention),
"parallel_2" (attention with biases beside retention) or "delta" (gated delta rule), its ``mixer``
sizes, and ``mlp``, ``kind`` "moe", or null.  model.safetensors holds the weights under the names of
:meth:`HybridConfig.tensor_shapes`; the inner size of the decay projection is that of its tensor.
"""
from __future__ import annotations

from .hybrid import (AttentionSpec, GatedDeltaSpec, GatedLinearSpec, HybridConfig, LayerSpec, MoESpec, PostNormForm,
                     RetentionSpec, Rotation, TwoSidedSpec)

ARCHITECTURE = "Gezozen"


def _rotation(r: dict) -> Rotation:
    s = r.get("scaling")
    return Rotation(float(r["base"]), int(r["dims"]),
                    None if s is None else tuple(float(s[k]) for k in ("factor", "original", "fast", "slow")))


def _sizes(m: dict, *keys) -> list:
    return [int(m[k]) for k in keys]


def _attention(m: dict, bias: bool) -> AttentionSpec:
    mask, cap = m.get("mask"), m.get("softcap")
    return AttentionSpec(*_sizes(m, "heads", "kv_heads", "dim", "vdim"), float(m["scale"]), _rotation(m["rot"]),
                         0 if mask is None else int(mask["size"]), 0.0 if cap is None else float(cap), bias)


def _mixer(entry: dict):
    kind, m = entry["type"], entry["mixer"]
    if kind == "delta":
        return GatedDeltaSpec(*_sizes(m, "heads", "kv_heads", "dim", "vdim", "conv"))
    if kind not in ("parallel", "parallel_2"):
        raise NotImplementedError(f"layer type {kind!r} is not supported (parallel, parallel_2, delta)")
    r = m["right"]
    sizes = _sizes(r, "heads", "dim", "vdim")
    right = (GatedLinearSpec(*sizes, float(r["tau"])) if kind == "parallel" else
             RetentionSpec(*sizes, tuple(float(d) for d in r["decay"]), _rotation(r["rot"])))
    return TwoSidedSpec(_attention(m["left"], kind == "parallel_2"), right, float(m["left_scale"]), float(m["right_scale"]))


def _mlp(m: dict | None) -> MoESpec | None:
    if m is None:
        return None
    if m["kind"] != "moe":
        raise NotImplementedError(f"feed-forward kind {m['kind']!r} is not supported (moe)")
    sh = m.get("shared")
    return MoESpec(int(m["router"]["experts"]), int(m["router"]["top"]), int(m["expert"]["ff"]), 0 if sh is None else int(sh["ff"]))


def config_from_json(js: dict, name: str = "gezozen") -> HybridConfig:
    return HybridConfig(name=name, vocab_size=int(js["vocab"]), hidden=int(js["width"]),
                        layer_specs=[LayerSpec(_mixer(e), moe=_mlp(e.get("mlp"))) for e in js["layers"]],
                        rms_eps=float(js["norm"]["eps"]),
                        post=PostNormForm(float(js["postln_alpha"]), int(js["norm"]["groups"])))


def config_to_json(cfg: HybridConfig) -> dict:
    def rot(r):
        out = {"base": r.base, "dims": r.dims}
        if r.scaling is not None:
            out["scaling"] = dict(zip(("factor", "original", "fast", "slow"), r.scaling))
        return out

    def attention(s):
        out = {"heads": s.heads, "kv_heads": s.kv_heads, "dim": s.dim, "vdim": s.vdim, "scale": s.scale, "rot": rot(s.rot)}
        if s.window:
            out["mask"] = {"size": s.window}
        if s.softcap:
            out["softcap"] = s.softcap
        return out

    layers = []
    for sp in cfg.layer_specs:
        m = sp.mixer
        if isinstance(m, GatedDeltaSpec):
            kind, mx = "delta", {"heads": m.heads, "kv_heads": m.kv_heads, "dim": m.dim, "vdim": m.vdim, "conv": m.conv}
        else:
            r = m.right
            right = {"heads": r.heads, "dim": r.dim, "vdim": r.vdim}
            gla = isinstance(r, GatedLinearSpec)
            kind = "parallel" if gla else "parallel_2"
            right.update({"tau": r.tau} if gla else {"decay": list(r.decay), "rot": rot(r.rot)})
            mx = {"left": attention(m.left), "right": right, "left_scale": m.left_scale, "right_scale": m.right_scale}
        f, mlp = sp.moe, None
        if f is not None:
            mlp = {"kind": "moe", "expert": {"ff": f.ff}, "router": {"experts": f.experts, "top": f.top}}
            if f.shared:
                mlp["shared"] = {"ff": f.shared}
        layers.append({"type": kind, "mixer": mx, "mlp": mlp})
    return {"architecture": ARCHITECTURE, "vocab": cfg.vocab_size, "width": cfg.hidden, "postln_alpha": cfg.post.alpha,
            "norm": {"eps": cfg.rms_eps, "groups": cfg.post.groups}, "layers": layers}


def _decays(n: int) -> tuple:
    """Retention's decays, 1 - 2^-5 to 1 - 2^-12 over the heads."""
    return tuple(1 - 2.0 ** -(5 + 7 * i / max(n - 1, 1)) for i in range(n))


def preset(name: str) -> HybridConfig:
    if name == "gezozen-tiny":        # kernel / engine / service tests
        moe = MoESpec(6, 2, 96, 64)
        a = TwoSidedSpec(AttentionSpec(4, 2, 32, 48, 0.18, Rotation(1e4, 16), 0, 30.0), GatedLinearSpec(2, 24, 40, 8.0, 12), 0.8, 1.0)
        b = TwoSidedSpec(AttentionSpec(4, 1, 24, 32, 0.2, Rotation(2e4, 24, (4.0, 512.0, 32.0, 1.0)), 80, 0.0, True),
                         RetentionSpec(3, 32, 24, _decays(3), Rotation(1e5, 32)), 1.0, 0.7)
        return HybridConfig(name=name, vocab_size=4096, hidden=192, post=PostNormForm(2.0, 3), layer_specs=[
            LayerSpec(a, moe=moe), LayerSpec(b, moe=moe), LayerSpec(GatedDeltaSpec(4, 2, 32, 40, 4), moe=moe)])
    if name == "gezozen-8b":          # the layer sizes of an 8B-class model
        moe = MoESpec(16, 2, 2048, 2048)
        d, half = 128, 64
        a = TwoSidedSpec(AttentionSpec(16, 4, d, d, d ** -0.5, Rotation(5e5, half), 0, 50.0), GatedLinearSpec(16, d, d, 16.0, 64), 1.0, 1.0)
        b = TwoSidedSpec(AttentionSpec(16, 4, d, d, d ** -0.5, Rotation(5e4, half, (8.0, 4096.0, 32.0, 1.0)), 1024, 0.0, True),
                         RetentionSpec(16, d, d, _decays(16), Rotation(1e6, d)), 1.0, 1.0)
        c = GatedDeltaSpec(32, 16, d, d, 4)
        return HybridConfig(name=name, vocab_size=128256, hidden=4096, post=PostNormForm(3.0, 4),
                            layer_specs=[LayerSpec(m, moe=moe) for m in (a, b, c, c) * 4])
    raise ValueError(f"unknown gezozen preset {name}")
