"""The Saritar decoder: its config.json, tensor names and presets, on models/hybrid.py.

config.json: ``architecture`` "Saritar", ``vocab``, ``width``, ``embedding.scale``,
``norm.eps``, ``layers`` (each ``type`` "attention" | "mamba1", ``mixer`` sizes and ``mlp``,
``kind`` "dense" with ``ff``, or null) and ``loop`` (``start``, ``stop``, ``times``: layers
start .. stop - 1 run ``times`` times over the same weights).  model.safetensors holds the
weights under the names of :meth:`HybridConfig.tensor_shapes`.
"""
from __future__ import annotations

from .hybrid import HybridConfig, LayerSpec, SelectiveScanSpec, WindowAttentionSpec

ARCHITECTURE = "Saritar"


def _mixer(entry: dict):
    kind, m = entry["type"], entry["mixer"]
    if kind == "attention":
        if m.get("vdim", m["dim"]) != m["dim"]:
            raise ValueError(f"attention values are the keys: vdim {m['vdim']} must equal dim {m['dim']}")
        return WindowAttentionSpec(int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), float(m["scale"]),
                                   int(m["mask"]["size"]))
    if kind == "mamba1":
        return SelectiveScanSpec(int(m["inner"]), int(m["state"]), int(m["dt_rank"]), int(m["conv"]))
    raise NotImplementedError(f"layer type {kind!r} is not supported (attention, mamba1)")


def config_from_json(js: dict, name: str = "saritar") -> HybridConfig:
    layers = []
    for e in js["layers"]:
        mlp = e.get("mlp")
        if mlp is not None and mlp["kind"] != "dense":
            raise NotImplementedError(f"feed-forward kind {mlp['kind']!r} is not supported (dense)")
        layers.append(LayerSpec(_mixer(e), int(mlp["ff"]) if mlp is not None else 0))
    lp = js.get("loop")
    return HybridConfig(name=name, vocab_size=int(js["vocab"]), hidden=int(js["width"]), layer_specs=layers,
                        embed_scale=float(js["embedding"]["scale"]), rms_eps=float(js["norm"]["eps"]),
                        loop=(int(lp["start"]), int(lp["stop"]), int(lp["times"])) if lp else None)


def config_to_json(cfg: HybridConfig) -> dict:
    layers = []
    for sp in cfg.layer_specs:
        m = sp.mixer
        if isinstance(m, WindowAttentionSpec):
            e = {"type": "attention", "mixer": {"heads": m.heads, "kv_heads": m.kv_heads, "dim": m.dim, "vdim": m.dim,
                                                "scale": m.scale, "mask": {"size": m.window}}}
        else:
            e = {"type": "mamba1", "mixer": {"inner": m.inner, "state": m.state, "dt_rank": m.dt_rank, "conv": m.conv}}
        e["mlp"] = {"kind": "dense", "ff": sp.ff} if sp.ff else None
        layers.append(e)
    return {"architecture": ARCHITECTURE, "vocab": cfg.vocab_size, "width": cfg.hidden,
            "embedding": {"scale": cfg.embed_scale}, "norm": {"eps": cfg.rms_eps}, "layers": layers,
            "loop": dict(zip(("start", "stop", "times"), cfg.loop)) if cfg.loop else None}


def preset(name: str) -> HybridConfig:
    if name == "saritar-tiny":        # kernel / engine / service tests
        att = LayerSpec(WindowAttentionSpec(4, 2, 32, 0.2, 48), 512)
        ssm = LayerSpec(SelectiveScanSpec(512, 16, 16, 4))
        return HybridConfig(name=name, vocab_size=4096, hidden=256, layer_specs=[ssm, att, ssm, ssm], embed_scale=2.0,
                            loop=(1, 3, 2))
    if name == "saritar-8b":          # the layer sizes of an 8B-class model, one attention layer in four
        att = LayerSpec(WindowAttentionSpec(32, 8, 128, 128 ** -0.5, 1024), 14336)
        ssm = LayerSpec(SelectiveScanSpec(8192, 16, 256, 4))
        return HybridConfig(name=name, vocab_size=128256, hidden=4096, layer_specs=[ssm, ssm, att, ssm] * 12,
                            embed_scale=1.0, loop=(4, 8, 2))
    raise ValueError(f"unknown saritar preset {name}")
