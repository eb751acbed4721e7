"""Gezozen on the CPU reference operators: configuration, checkpoint IO, registry, engine,
scheduler and command line against the plain oracle."""
import copy
import json
import subprocess
import sys
from pathlib import Path

import pytest
import torch

sys.path.insert(0, str(Path(__file__).parent))
import gezozen_cases as C  # noqa: E402
import gezozen_oracle as O  # noqa: E402

ROOT = Path(__file__).resolve().parent.parent
F32 = torch.float32


@pytest.fixture(autouse=True)
def _threads():
    n = torch.get_num_threads()
    torch.set_num_threads(2)          # tiny operators: more threads only contend
    yield
    torch.set_num_threads(n)


def test_rotation():
    C.rope_case("cpu")


@pytest.mark.parametrize("case", ["post_norm_case", "attention_case", "window_edge_case", "soft_cap_case", "batch_attention_case",
                                  "linear_case", "decay_case", "batch_linear_case", "forgotten_state_case", "conv_case", "moe_case"])
def test_mechanisms(case):
    getattr(C, case)("cpu", F32)


@pytest.mark.parametrize("name", list(C.CONFIGS))
def test_models(name):
    C.whole_case(name, "cpu", F32)
    C.portions_case(name, "cpu", F32, T=61 if name != "edge" else 90)
    C.batch_case(name, "cpu", F32)


def test_settled_routing_in_bf16():
    for name in C.CONFIGS:
        C.whole_case(name, "cpu", torch.bfloat16)


def test_long_decoding():
    C.long_case("edge", "cpu", F32)


@pytest.mark.parametrize("name", ["mixed", "odd"])
def test_generation(name):
    C.generate_case(name, "cpu")
    C.mixed_steps_case(name, "cpu")


def test_preemption_recomputes_state():
    C.preemption_case("mixed", "cpu")


def test_a_mistake_in_the_oracle_shows(monkeypatch):
    """The comparisons see what they are meant to see: an oracle with one wrong constant, window
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

    wrong(lambda d: mx(d, 1)["left"]["mask"].update(size=10))
    wrong(lambda d: mx(d, 1)["left"]["rot"]["scaling"].update(factor=5.0))
    wrong(lambda d: mx(d, 1)["left"]["rot"].pop("scaling"))
    wrong(lambda d: mx(d, 0)["left"]["rot"].update(base=9e3))
    wrong(lambda d: mx(d, 0)["left"].update(softcap=7.0))
    wrong(lambda d: mx(d, 0)["left"].update(scale=0.28))
    wrong(lambda d: mx(d, 0)["right"].update(tau=5.0))
    wrong(lambda d: mx(d, 1)["right"]["rot"].update(base=9e4))
    wrong(lambda d: mx(d, 1)["right"]["decay"].reverse())
    wrong(lambda d: mx(d, 0).update(left_scale=0.75))
    wrong(lambda d: mx(d, 1).update(right_scale=0.9))
    wrong(lambda d: d["norm"].update(eps=3e-3))
    wrong(lambda d: d["norm"].update(groups=2))
    wrong(lambda d: d.update(postln_alpha=2.6))
    wrong(lambda d: d["layers"][0]["mlp"]["router"].update(top=1))
    wrong(lambda d: d["layers"][2]["mlp"].pop("shared"))
    for name in ("l0.rg1.b", "l1.rg2", "l2.norm1", "l0.mix.left.q.norm", "l1.mix.left.v.b", "l0.mix.right.a2.b", "l0.mix.right.norm",
                 "l2.mix.A_log", "l2.mix.dt_bias", "l2.mix.k.conv", "l2.mix.b", "l2.mix.norm", "l2.mlp.shared.sg", "l1.mlp.router"):
        wrong(weights={k: v + 0.1 if k == name else v for k, v in w.items()})
    # the weight on the expert's output instead of its input; a read-out that misses the current write
    monkeypatch.setattr(O, "expert", lambda h, t, f=O.expert: f(h, t) * 0.9)
    wrong()
    monkeypatch.undo()
    monkeypatch.setattr(O, "unit", lambda x: x)
    wrong()


def test_config_round_trip_and_refusals():
    from docqa_amd.models import gezozen

    for js in C.CONFIGS.values():
        cfg = gezozen.config_from_json(js)
        assert gezozen.config_to_json(cfg) == js
        want = cfg.tensor_shapes()
        for k, v in O.random_weights(js).items():
            s = want.pop(k)
            assert len(s) == v.dim() and all(n in (0, m) for n, m in zip(s, v.shape)), k
        assert not want
    base = json.dumps(C.CONFIGS["mixed"])
    mx = lambda d, i: d["layers"][i]["mixer"]  # noqa: E731
    for bad in (lambda d: d["layers"][0].update(type="attention"), lambda d: d["layers"][0]["mlp"].update(kind="dense"),
                lambda d: mx(d, 0)["left"].update(kv_heads=3), lambda d: mx(d, 0)["left"]["rot"].update(dims=18),
                lambda d: mx(d, 0)["left"]["rot"].update(dims=7), lambda d: mx(d, 1)["right"].update(decay=[0.5]) or mx(d, 1)["right"].update(heads=2),
                lambda d: mx(d, 1)["right"].update(decay=[0.5, 1.5]), lambda d: mx(d, 2).update(kv_heads=3), lambda d: mx(d, 2).update(conv=0),
                lambda d: mx(d, 0)["right"].update(tau=0.0), lambda d: d["norm"].update(groups=7),
                lambda d: d["layers"][0]["mlp"]["router"].update(top=6), lambda d: mx(d, 2).update(dim=300)):
        d = json.loads(base)
        bad(d)
        with pytest.raises((ValueError, NotImplementedError)):
            gezozen.config_from_json(d)


def test_caches_of_a_layer():
    """A mixer of two sides has a paged cache and a state, a delta layer a state alone."""
    js, w, m = C.make("mixed", "cpu", F32)
    eng = C.engine(m)
    assert [(k.shape[1], k.shape[3], v.shape[3]) for k, v in eng.kv.caches] == [(2, 16, 24), (1, 24, 16)]
    assert [tuple(tuple(t.shape[1:]) for t in s) for s in eng.state.states] == [
        ((3, 16, 24),), ((2, 16, 8),), ((3, 2 * 16 * 2 + 4 * 24), (4, 16, 24))]
    assert all(t.dtype == F32 for s in eng.state.states for t in s)
    bf = C.engine(C.make("mixed", "cpu", torch.bfloat16)[2]).state.states
    assert [[t.dtype for t in s] for s in bf] == [[F32], [F32], [torch.bfloat16, F32]]


def _save(tmp_path, name="mixed"):
    from docqa_amd.models import checkpoint as ck
    from docqa_amd.models import gezozen

    js = C.CONFIGS[name]
    w = O.random_weights(js, 31)
    ck.save_gezozen(gezozen.config_from_json(js), w, tmp_path / name)
    return js, w, tmp_path / name


def test_registry_and_checkpoint(tmp_path):
    from docqa_amd.models import checkpoint as ck
    from docqa_amd.models.hybrid import HybridModel

    js, w, d = _save(tmp_path)
    m = ck.resolve_decoder(d, device="cpu", dtype=F32)
    assert isinstance(m, HybridModel) and ck.decoder_family(d).name == "gezozen"
    seq = C.toks(20, js["vocab"], 2)
    C.close(C.run_steps(C.engine(m), [[("a", seq)]])["a"], O.forward(js, w, seq))
    m = ck.resolve_decoder("gezozen-tiny", device="cpu", dtype=F32, seed=3)
    assert isinstance(m, HybridModel) and m.cfg.name == "gezozen-tiny"
    cfg = json.loads((d / "config.json").read_text())
    cfg["layers"][0]["mlp"]["shared"]["ff"] += 1
    (d / "config.json").write_text(json.dumps(cfg))
    with pytest.raises(ValueError, match="shared"):
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


def test_qa_stack_over_gezozen():
    """The RAG pipeline runs with this generator named by its preset."""
    from docqa_amd.pipeline.builder import StackConfig, build_stack

    pipe, _ = build_stack(StackConfig(llm="gezozen-tiny", embed="tiny-bert", n_notes=20, max_batch=2, max_context=1024,
                                      use_graphs=False), device="cpu")
    pipe.answer("Which antibiotic was started?", C.SamplingParams(max_new_tokens=3, stop_on_eos=False))
    assert pipe.engine.state.num_free() == pipe.engine.state.slots
