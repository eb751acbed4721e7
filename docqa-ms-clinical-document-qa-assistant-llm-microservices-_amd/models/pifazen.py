"""The Pifazen decoder: its config.json, tensor names and presets, on models/hybrid.py.

config.json: ``architecture`` "Pifazen", ``vocab``, ``width``, ``norm`` (``eps``) and ``layers``:
``type`` "channel_delta" (gated delta rule with channel decays), "latent_attention" (queries through
a latent, a gate an output element) or "latent_attention_2" (YaRN rotation, a gate a head), its
``mixer`` sizes, ``mlp``, ``kind`` "dense" (PolyNorm) or "moe", or null, and ``weights_of`` where the
layer uses another's weights.  model.safetensors holds the weights under the names of
:meth:`HybridConfig.tensor_shapes`; the inner sizes of a delta layer's decay and gate projections are
those of their tensors.
"""
from __future__ import annotations

from .. import ops
from .hybrid import (ChannelDeltaSpec, GroupRouter, HybridConfig, LatentAttentionSpec, LayerSpec, MoESpec, PreNormForm)

ARCHITECTURE = "Pifazen"
_SCALING = ("factor", "original", "fast", "slow")


def _sizes(m: dict, *keys) -> list:
    return [int(m[k]) for k in keys]


def _latent(heads, dim, rot_dim, vdim, kv_rank, scale, base, q_rank=0, scaling=None, gate="head") -> LatentAttentionSpec:
    """What the design fixes: no window, no sink, rotated neighbours, an output gate."""
    return LatentAttentionSpec(heads, dim, rot_dim, vdim, kv_rank, scale, 0, base, scaling=scaling, interleaved=True, q_rank=q_rank,
                               gate=gate, sink=False)


def _mixer(entry: dict):
    kind, m = entry["type"], entry["mixer"]
    if kind == "channel_delta":
        return ChannelDeltaSpec(*_sizes(m, "heads", "kv_heads", "dim", "vdim", "conv"))
    if kind not in ("latent_attention", "latent_attention_2"):
        raise NotImplementedError(f"layer type {kind!r} is not supported (channel_delta, latent_attention, latent_attention_2)")
    r = m["rot"]
    if r["dims"] != m["rot_dim"]:
        raise ValueError(f"rot.dims {r['dims']} must be the rotated part, rot_dim {m['rot_dim']}")
    s = r.get("scaling")
    first = kind == "latent_attention"
    return _latent(*_sizes(m, "heads", "dim", "rot_dim", "vdim", "kv_rank"), float(m["scale"]), float(r["base"]),
                   int(m["q_rank"]) if first else 0, None if s is None else tuple(float(s[k]) for k in _SCALING),
                   "element" if first else "head")


def _mlp(m: dict | None) -> dict:
    if m is None:
        return {}
    if m["kind"] == "dense":
        return {"ff": int(m["ff"])}
    if m["kind"] != "moe":
        raise NotImplementedError(f"feed-forward kind {m['kind']!r} is not supported (dense, moe)")
    r = m["router"]
    g = r.get("groups") or {"count": 1, "keep": 1}
    router = GroupRouter(int(r.get("identity") or 0), *_sizes(g, "count", "keep"), float(r.get("scale", 1.0)))
    return {"moe": MoESpec(int(r["experts"]), int(r["top"]), int(m["expert"]["ff"]), router=router, limit=float(m["expert"]["limit"]))}


def _owner(layers: list, i: int) -> int | None:
    """The layer whose tensors layer i uses, if not its own."""
    j, seen = layers[i].get("weights_of"), set()
    while j is not None and 0 <= j < len(layers) and layers[j].get("weights_of") is not None and j not in seen:
        seen.add(j)
        j = layers[j]["weights_of"]
    return None if j is None else int(j)


def _config(name: str, **kw) -> HybridConfig:
    """What the design fixes: norm weights stored around zero, PolyNorm, the embedding as LM head."""
    return HybridConfig(name=name, pre=PreNormForm(), tied=True, act=ops.ACT_POLY_NORM, norm_offset=1.0, **kw)


def config_from_json(js: dict, name: str = "pifazen") -> HybridConfig:
    layers = js["layers"]
    specs = [LayerSpec(_mixer(e), **_mlp(e.get("mlp")), weights_of=_owner(layers, i)) for i, e in enumerate(layers)]
    return _config(name, vocab_size=int(js["vocab"]), hidden=int(js["width"]), layer_specs=specs, rms_eps=float(js["norm"]["eps"]))


def config_to_json(cfg: HybridConfig) -> dict:
    layers = []
    for sp in cfg.layer_specs:
        m, f, mlp = sp.mixer, sp.moe, None
        if isinstance(m, ChannelDeltaSpec):
            kind, mx = "channel_delta", {k: getattr(m, k) for k in ("heads", "kv_heads", "dim", "vdim", "conv")}
        else:
            kind = "latent_attention" if m.gate == "element" else "latent_attention_2"
            mx = {k: getattr(m, k) for k in ("heads", "dim", "rot_dim", "vdim", "kv_rank", "scale")}
            mx["rot"] = {"base": m.rope_base, "dims": m.rot_dim}
            if m.scaling is not None:
                mx["rot"]["scaling"] = dict(zip(_SCALING, m.scaling))
            if m.q_rank:
                mx["q_rank"] = m.q_rank
        if sp.ff:
            mlp = {"kind": "dense", "ff": sp.ff}
        elif f is not None:
            r = f.router
            mlp = {"kind": "moe", "expert": {"ff": f.ff, "limit": f.limit},
                   "router": {"experts": f.experts, "identity": r.identity, "top": f.top, "scale": r.scale,
                              "groups": {"count": r.groups, "keep": r.keep}}}
        layers.append({"type": kind, "mixer": mx, "mlp": mlp})
        if sp.weights_of is not None:
            layers[-1]["weights_of"] = sp.weights_of
    return {"architecture": ARCHITECTURE, "vocab": cfg.vocab_size, "width": cfg.hidden, "norm": {"eps": cfg.rms_eps}, "layers": layers}


def preset(name: str) -> HybridConfig:
    yarn = (8.0, 4096.0, 32.0, 1.0)
    if name == "pifazen-tiny":        # kernel / engine / service tests
        a = _latent(4, 24, 8, 40, 48, 0.18, 1e4, 56, gate="element")
        b = _latent(3, 32, 16, 24, 72, 0.15, 2e4, scaling=(4.0, 512.0, 32.0, 1.0))
        c = ChannelDeltaSpec(4, 2, 32, 40, 4, 12, 20)
        moe = MoESpec(6, 2, 96, router=GroupRouter(2, 4, 2, 1.5), limit=3.0)
        return _config(name, vocab_size=4096, hidden=192, rms_eps=1e-5, layer_specs=[
            LayerSpec(a, 256), LayerSpec(c, moe=moe), LayerSpec(b, moe=moe), LayerSpec(c, moe=moe, weights_of=1)])
    if name == "pifazen-8b":          # the layer sizes of an 8B-class model
        a = _latent(32, 128, 64, 128, 512, 192 ** -0.5, 5e5, 1536, gate="element")
        b = _latent(32, 128, 64, 128, 512, 192 ** -0.5, 1e6, scaling=yarn)
        c = ChannelDeltaSpec(32, 32, 128, 128, 4, 128, 128)
        moe = MoESpec(16, 3, 2048, router=GroupRouter(2, 3, 2, 2.0), limit=7.0)
        return _config(name, vocab_size=128256, hidden=4096, rms_eps=1e-5, layer_specs=[LayerSpec(c, 14336)] + [
            LayerSpec(m, moe=moe) for m in (c, c, a) + (c, c, c, b) + (c, c, c, a) + (c, c, c, b)])
    raise ValueError(f"unknown pifazen preset {name}")
