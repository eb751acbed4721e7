"""The Dolodra decoder: its config.json, tensor names and presets, on models/hybrid.py.

config.json: ``architecture`` "Dolodra", ``vocab``, ``width``, ``embedding.scale``,
``norm.eps``, ``residual_mult``, ``logit_softcap``, ``canon.taps``, ``token_side.dim`` and
``layers`` (each ``type`` "latent_attention", its ``mixer`` sizes -- ``kv_from`` where it reads
another layer's latents -- and ``mlp``, ``kind`` "dense" with ``ff``, or null).
model.safetensors holds the weights under the names of :meth:`HybridConfig.tensor_shapes`.
"""
from __future__ import annotations

from .. import ops
from .hybrid import HybridConfig, LatentAttentionSpec, LayerSpec, ParallelForm

ARCHITECTURE = "Dolodra"


def _mixer(entry: dict) -> LatentAttentionSpec:
    kind, m = entry["type"], entry["mixer"]
    if kind != "latent_attention":
        raise NotImplementedError(f"layer type {kind!r} is not supported (latent_attention)")
    if m["rot"]["dims"] != m["rot_dim"]:
        raise ValueError(f"rot.dims {m['rot']['dims']} must be the rotated part, rot_dim {m['rot_dim']}")
    src = m.get("kv_from")
    return LatentAttentionSpec(int(m["heads"]), int(m["dim"]), int(m["rot_dim"]), int(m["vdim"]), int(m["kv_rank"]),
                               float(m["scale"]), int(m["mask"]["size"]), float(m["rot"]["base"]),
                               None if src is None else int(src))


def _config(name: str, parallel: ParallelForm, cap: float, **kw) -> HybridConfig:
    """What the design fixes: tanh GELU, norm weights stored around zero."""
    return HybridConfig(name=name, parallel=parallel, act=ops.ACT_GELU_TANH, norm_offset=1.0, logit_softcap=cap, **kw)


def config_from_json(js: dict, name: str = "dolodra") -> HybridConfig:
    layers = []
    for e in js["layers"]:
        mlp = e.get("mlp")
        if mlp is not None and mlp["kind"] != "dense":
            raise NotImplementedError(f"feed-forward kind {mlp['kind']!r} is not supported (dense)")
        layers.append(LayerSpec(_mixer(e), int(mlp["ff"]) if mlp is not None else 0))
    par = ParallelForm(float(js["residual_mult"]), int(js["canon"]["taps"]), int(js["token_side"]["dim"]))
    return _config(name, par, float(js["logit_softcap"]), vocab_size=int(js["vocab"]), hidden=int(js["width"]),
                   layer_specs=layers, embed_scale=float(js["embedding"]["scale"]), rms_eps=float(js["norm"]["eps"]))


def config_to_json(cfg: HybridConfig) -> dict:
    layers = []
    for sp in cfg.layer_specs:
        m = sp.mixer
        mx = {"heads": m.heads, "dim": m.dim, "rot_dim": m.rot_dim, "vdim": m.vdim, "kv_rank": m.kv_rank,
              "scale": m.scale, "mask": {"size": m.window}, "rot": {"base": m.rope_base, "dims": m.rot_dim}}
        if m.kv_from is not None:
            mx["kv_from"] = m.kv_from
        layers.append({"type": "latent_attention", "mixer": mx, "mlp": {"kind": "dense", "ff": sp.ff} if sp.ff else None})
    par = cfg.parallel
    return {"architecture": ARCHITECTURE, "vocab": cfg.vocab_size, "width": cfg.hidden,
            "embedding": {"scale": cfg.embed_scale}, "norm": {"eps": cfg.rms_eps}, "residual_mult": par.mult,
            "logit_softcap": cfg.logit_softcap, "canon": {"taps": par.conv}, "token_side": {"dim": par.side},
            "layers": layers}


def preset(name: str) -> HybridConfig:
    if name == "dolodra-tiny":        # kernel / engine / service tests
        own = LayerSpec(LatentAttentionSpec(4, 24, 8, 40, 64, 0.2, 48, 1e4), 384)
        return _config(name, ParallelForm(0.5, 3, 24), 20.0, vocab_size=4096, hidden=192, embed_scale=8.0, rms_eps=1e-5,
                       layer_specs=[own, LayerSpec(LatentAttentionSpec(6, 16, 8, 24, 64, 0.2, 96, 1e4, 0), 256), own])
    if name == "dolodra-8b":          # the layer sizes of an 8B-class model, every other layer on shared latents
        mx = (32, 128, 64, 128, 512, 192 ** -0.5, 1024, 5e5)
        layers = [LayerSpec(LatentAttentionSpec(*mx, None if i % 2 == 0 else i - 1), 14336) for i in range(32)]
        return _config(name, ParallelForm(0.25, 4, 256), 30.0, vocab_size=128256, hidden=4096, embed_scale=64.0,
                       rms_eps=1e-5, layer_specs=layers)
    raise ValueError(f"unknown dolodra preset {name}")
