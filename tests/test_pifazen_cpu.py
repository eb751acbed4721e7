"""Pifazen on the CPU reference operators: configuration, checkpoint IO, registry, engine,
scheduler and command line against the plain oracle."""
import copy
import json
import subprocess
import sys
from pathlib import Path

import pytest
import torch

sys.path.insert(0, str(Path(__file__).parent))
import pifazen_cases as C  # noqa: E402
import pifazen_oracle as O  # noqa: E402

ROOT = Path(__file__).resolve().parent.parent
F32 = torch.float32
MECHANISMS = ["scaled_norm_case", "mix_case", "poly_norm_case", "query_latent_case", "head_gate_case", "latent_layer_case", "far_case", "delta_case",
              "delta_decay_case", "delta_batch_case", "forgotten_state_case", "low_rank_case", "delta_layer_case", "moe_case", "group_case",
              "clamp_case"]


@pytest.fixture(autouse=True)
def _threads():
    n = torch.get_num_threads()
    torch.set_num_threads(2)          # tiny operators: more threads only contend
    yield
    torch.set_num_threads(n)


@pytest.mark.parametrize("case", MECHANISMS)
def test_mechanisms(case):
    getattr(C, case)("cpu", F32)


@pytest.mark.parametrize("name", list(C.CONFIGS))
def test_models(name):
    C.MODELS.whole(name, "cpu", F32)
    C.MODELS.portions(name, "cpu", F32, T=61 if name != "edge" else 90)
    C.MODELS.batch(name, "cpu", F32)


def test_settled_routing_in_bf16():
    for name in ("mixed", "odd", "edge"):          # (the norm of one element is a sign: "ones" runs in fp32)
        C.MODELS.whole(name, "cpu", torch.bfloat16)


def test_long_decoding():
    C.MODELS.long("edge", "cpu", F32)


@pytest.mark.parametrize("name", ["mixed", "odd"])
def test_generation(name):
    C.MODELS.generate(name, "cpu")
    C.MODELS.mixed_steps(name, "cpu")


def test_preemption_recomputes_state():
    C.MODELS.preemption("mixed", "cpu")


def test_a_model_without_recurrence():
    """Attention layers alone: caches and no state."""
    js = C.conf(48, 53, [C.lat(2, 8, 8, 8, 16, 24, mlp=C.dense(32)), C.lat2(2, 8, 4, 8, 16, C.YARN)])
    C.MODELS.batch(js, "cpu", F32)
    C.MODELS.generate(js, "cpu")


def test_a_mistake_in_the_oracle_shows(monkeypatch):
    """The comparisons see what they are meant to see: an oracle with one wrong constant, weight
    or mechanism differs by many times the tolerance."""
    js, w, m = C.make("mixed", "cpu", F32)
    seq = C.toks(45, js["vocab"], 1)
    got = C.run_steps(C.engine(m), [[("a", seq)]])["a"]

    def wrong(change=lambda d: None, weights=w):
        d = copy.deepcopy(js)
        change(d)
        with pytest.raises(AssertionError):
            C.close(got, O.forward(d, weights, seq))

    def mx(d, i):
        return d["layers"][i]["mixer"]

    def router(d, i):
        return d["layers"][i]["mlp"]["router"]

    wrong(lambda d: mx(d, 2)["rot"]["scaling"].update(factor=5.0))
    wrong(lambda d: mx(d, 2)["rot"].pop("scaling"))
    wrong(lambda d: mx(d, 0)["rot"].update(base=9e3))
    wrong(lambda d: mx(d, 0).update(scale=0.26))
    wrong(lambda d: d["norm"].update(eps=1e-3))
    wrong(lambda d: router(d, 1).update(top=2))
    wrong(lambda d: router(d, 1).update(scale=1.6))
    wrong(lambda d: router(d, 1)["groups"].update(keep=3))
    wrong(lambda d: router(d, 2)["groups"].update(keep=2))
    wrong(lambda d: d["layers"][1]["mlp"]["expert"].update(limit=1.0))
    wrong(lambda d: d["layers"][3].update(weights_of=1, mlp=None))
    for name in ("l0.norm1", "l0.ls1", "l1.ls2", "l2.norm2", "l0.mix.dq.norm", "l0.mix.g", "l2.mix.g", "l2.mix.dkv.norm", "l0.mlp.up.b", "l0.mlp.down.b",
                 "l0.mlp.act", "l1.mix.A_log", "l1.mix.dt_bias", "l1.mix.a1", "l1.mix.g2", "l1.mix.k.conv", "l1.mix.b", "l1.mix.norm",
                 "final.norm"):
        wrong(weights={k: v + 0.1 if k == name else v for k, v in w.items()})
    for name in ("l1.mlp.correction", "l2.mlp.router"):
        wrong(weights={k: v.flip(0) if k == name else v for k, v in w.items()})
    for name, bad in (("rotate", lambda x, r, f=O.rotate: f(x.unflatten(-1, (2, -1)).mT.flatten(-2), r)), ("unit", lambda x: x),
                      ("layer_norm", lambda x, w, eps: O.unit_rms(x, eps) * w), ("channel_decay", lambda h, t, H, d, f=O.channel_decay: f(h, t, H, d).mean(-1, keepdim=True).expand(-1, -1, d)),
                      ("expert", lambda h, t, limit, f=O.expert: f(h, t, limit) * 0.9)):
        monkeypatch.setattr(O, name, bad)
        wrong()
        monkeypatch.undo()


def test_config_round_trip_and_refusals():
    from docqa_amd.models import pifazen

    for js in C.CONFIGS.values():
        cfg = pifazen.config_from_json(js)
        assert pifazen.config_to_json(cfg) == js
        want = cfg.tensor_shapes()
        for k, v in O.random_weights(js).items():
            s = want.pop(k)
            assert len(s) == v.dim() and all(n in (0, m) for n, m in zip(s, v.shape)), k
        assert not want
    base = json.dumps(C.CONFIGS["mixed"])
    mx = lambda d, i: d["layers"][i]["mixer"]  # noqa: E731
    rt = lambda d, i: d["layers"][i]["mlp"]["router"]  # noqa: E731
    for bad in (lambda d: d["layers"][0].update(type="attention"), lambda d: d["layers"][0]["mlp"].update(kind="sparse"),
                lambda d: mx(d, 1).update(kv_heads=3), lambda d: mx(d, 0)["rot"].update(dims=6), lambda d: mx(d, 0).update(rot_dim=7, rot=C.rot(1e4, 7)),
                lambda d: mx(d, 1).update(conv=0), lambda d: mx(d, 1).update(dim=300), lambda d: rt(d, 1).update(top=5), lambda d: rt(d, 1)["groups"].update(count=3),
                lambda d: rt(d, 1)["groups"].update(keep=5), lambda d: d["layers"][1]["mlp"]["expert"].update(limit=0.0),
                lambda d: d["layers"][3].update(weights_of=0), lambda d: d["layers"][3].update(weights_of=3), lambda d: d["layers"][3].update(weights_of=9),
                lambda d: d["layers"][3].update(mlp=None)):
        d = json.loads(base)
        bad(d)
        with pytest.raises((ValueError, NotImplementedError)):
            pifazen.config_from_json(d)
    # a layer may use one that uses another's, and one that comes after it
    d = json.loads(base)
    d["layers"].append(dict(d["layers"][3], weights_of=3))
    d["layers"].insert(0, dict(d["layers"][1], weights_of=2))
    for L in d["layers"][1:]:
        if "weights_of" in L:
            L["weights_of"] += 1
    assert [s.weights_of for s in pifazen.config_from_json(d).layer_specs] == [2, None, None, None, 2, None, 2]


def test_caches_of_a_layer():
    """A latent layer keeps one row a token, a delta layer convolution inputs and a state; a layer on another's
    weights keeps its own, and its owner's tensors."""
    js, w, m = C.make("mixed", "cpu", F32)
    eng = C.engine(m)
    assert [(k.shape[1], k.shape[3], v) for k, v in eng.kv.caches] == [(1, 48, None), (1, 48, None), (1, 32, None)]
    assert [tuple(tuple(t.shape[1:]) for t in s) for s in eng.state.states] == [((3, 2 * 32 + 96), (4, 16, 24))] * 2
    assert m.layers[1] is m.layers[3] and m.lm_head is m.embed
    bf = C.engine(C.make("mixed", "cpu", torch.bfloat16)[2]).state.states
    assert [[t.dtype for t in s] for s in bf] == [[torch.bfloat16, F32]] * 2


def _save(tmp_path, name="mixed"):
    from docqa_amd.models import checkpoint as ck
    from docqa_amd.models import pifazen

    js = C.CONFIGS[name]
    w = O.random_weights(js, 31)
    ck.save_pifazen(pifazen.config_from_json(js), w, tmp_path / name)
    return js, w, tmp_path / name


def test_registry_and_checkpoint(tmp_path):
    from docqa_amd.models import checkpoint as ck
    from docqa_amd.models.hybrid import HybridModel

    js, w, d = _save(tmp_path)
    m = ck.resolve_decoder(d, device="cpu", dtype=F32)
    assert isinstance(m, HybridModel) and ck.decoder_family(d).name == "pifazen"
    seq = C.toks(20, js["vocab"], 2)
    C.close(C.run_steps(C.engine(m), [[("a", seq)]])["a"], O.forward(js, w, seq))
    m = ck.resolve_decoder("pifazen-tiny", device="cpu", dtype=F32, seed=3)
    assert isinstance(m, HybridModel) and m.cfg.name == "pifazen-tiny"
    assert ck.resolve_decoder_config("pifazen-8b").num_params() > 4e9
    cfg = json.loads((d / "config.json").read_text())
    cfg["layers"][0]["mixer"]["q_rank"] += 1
    (d / "config.json").write_text(json.dumps(cfg))
    with pytest.raises(ValueError, match="mix.dq"):
        ck.resolve_decoder(d, device="cpu")


def test_trace_command(tmp_path):
    """bin/trace_run over a saved checkpoint: step files, their order and the exit code."""
    js, w, d = _save(tmp_path)
    a, b = C.toks(30, js["vocab"], 1), C.toks(12, js["vocab"], 2)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:20], "want": [0, 19]}], "end": []},
             {"step": 1, "entries": [{"id": "b", "tokens": b[:11], "want": []}], "end": []},
             {"step": 2, "entries": [{"id": "b", "tokens": b[11:], "want": [0]},
                                     {"id": "a", "tokens": a[20:], "want": [2, 9]}], "end": ["a", "b"]},
             {"step": 3, "entries": [{"id": "c", "tokens": b, "want": [11]}], "end": ["c"]}]
    r = subprocess.run([sys.executable, str(ROOT / "bin" / "trace_run"), "--model", str(d), "--dtype", "float32", "--out",
                        str(tmp_path / "out"), "--max-tokens", "128", "--device", "cpu"],
                       input="".join(json.dumps(s) + "\n" for s in steps), capture_output=True, text=True, timeout=120)
    assert r.returncode == 0, r.stderr
    assert [x for x in r.stdout.splitlines() if x.startswith("done")] == [f"done {i}" for i in range(4)]
    wa, wb = O.forward(js, w, a), O.forward(js, w, b)

    def logits(n):
        return torch.frombuffer(bytearray((tmp_path / "out" / f"{n}.f32").read_bytes()), dtype=F32).view(-1, js["vocab"])

    C.close(logits(0), wa[[0, 19]])
    C.close(logits(2), torch.stack([wb[11], wa[22], wa[29]]))
    C.close(logits(3), wb[11:])
    assert not (tmp_path / "out" / "1.f32").exists()


def test_qa_stack_over_pifazen():
    """The RAG pipeline runs with this generator named by its preset."""
    from docqa_amd.engine.llm_engine import SamplingParams
    from docqa_amd.pipeline.builder import StackConfig, build_stack

    pipe, _ = build_stack(StackConfig(llm="pifazen-tiny", embed="tiny-bert", n_notes=20, max_batch=2, max_context=1024,
                                      use_graphs=False), device="cpu")
    pipe.answer("Which antibiotic was started?", SamplingParams(max_new_tokens=3, stop_on_eos=False))
    assert pipe.engine.state.num_free() == pipe.engine.state.slots
