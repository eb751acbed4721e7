"""Saritar on the CPU reference operators: configuration, checkpoint IO, registry, engine,
scheduler and command line against the plain oracle."""
import json
import subprocess
import sys
from pathlib import Path

import pytest
import torch

sys.path.insert(0, str(Path(__file__).parent))
import saritar_cases as C  # noqa: E402
import saritar_oracle as O  # noqa: E402

ROOT = Path(__file__).resolve().parent.parent
F32 = torch.float32


@pytest.fixture(autouse=True)
def _threads():
    n = torch.get_num_threads()
    torch.set_num_threads(2)          # tiny operators: more threads only contend
    yield
    torch.set_num_threads(n)


def test_norms_and_activations():
    C.norm_case("cpu")
    C.embed_case("cpu")
    C.squared_relu_case("cpu")
    C.slab_columns_case("cpu")
    C.relu2_linear_case("cpu", [(3, 8, 16)])


@pytest.mark.parametrize("case", ["window_edge_case", "sink_case", "general_attention_case", "batch_attention_case",
                                  "conv_case", "scan_batch_case"])
def test_mechanisms(case):
    getattr(C, case)("cpu", F32)


def test_scan():
    C.scan_case("cpu", F32, ((24, 5, 40), (7, 1, 33), (9, 70, 18)))


@pytest.mark.parametrize("name", list(C.CONFIGS))
def test_whole_prompt(name):
    C.whole_case(name, "cpu", F32)


@pytest.mark.parametrize("name", ["mixed", "ones", "edge"])
def test_portions(name):
    C.portions_case(name, "cpu", F32, T=37)


@pytest.mark.parametrize("name", ["mixed", "attention", "recurrent"])
def test_batches(name):
    C.batch_case(name, "cpu", F32)


def test_far_tokens():
    C.far_case("cpu", F32)


@pytest.mark.parametrize("name", ["mixed", "attention"])
def test_generation(name):
    C.generate_case(name, "cpu")
    C.mixed_steps_case(name, "cpu")


def test_preemption_recomputes_state():
    C.preemption_case("mixed", "cpu")


def test_state_pool():
    C.state_pool_case()


def test_lagged_readback_frees_the_slot_once():
    """The GPU's readback order: a finished request rides one extra step on its slot."""
    js, w, m = C.make("mixed", "cpu", F32, seed=23)
    prompts = [C.toks(n, js["vocab"], n) for n in (6, 11, 3, 8)]
    ce = C.ContinuousEngine(C.engine(m, tokens=256, slots=2))
    ce.lag_cpu, ce.pad_buckets = True, True
    got = ce.generate(prompts, C.SamplingParams(max_new_tokens=5))
    assert got == [C.greedy_oracle(js, w, p, 5) for p in prompts]
    while ce.has_work():
        ce.step()
    assert ce.eng.state.num_free() == 2


def test_config_round_trip_and_refusals():
    from docqa_amd.models import saritar

    for js in C.CONFIGS.values():
        cfg = saritar.config_from_json(js)
        assert saritar.config_to_json(cfg) == js
        assert cfg.runs == O.runs_of(len(js["layers"]), js["loop"])
        assert {k: tuple(v.shape) for k, v in O.random_weights(js).items()} == cfg.tensor_shapes()
    base = json.dumps(C.CONFIGS["plain"])
    for bad in (lambda d: d["layers"][0].update(type="rwkv"), lambda d: d["layers"][0]["mlp"].update(kind="moe"),
                lambda d: d["layers"][0]["mixer"].update(vdim=5), lambda d: d["layers"][0]["mixer"].update(kv_heads=2),
                lambda d: d.update(loop={"start": 1, "stop": 9, "times": 2})):
        d = json.loads(base)
        bad(d)
        with pytest.raises((ValueError, NotImplementedError)):
            saritar.config_from_json(d)


def _save(tmp_path, name="mixed"):
    from docqa_amd.models import checkpoint as ck
    from docqa_amd.models import saritar

    js = C.CONFIGS[name]
    w = O.random_weights(js, 31)
    ck.save_saritar(saritar.config_from_json(js), w, tmp_path / name)
    return js, w, tmp_path / name


def test_registry_and_checkpoint(tmp_path):
    from docqa_amd.models import checkpoint as ck
    from docqa_amd.models.hybrid import HybridModel
    from docqa_amd.models.llama import LlamaModel

    js, w, d = _save(tmp_path)
    m = ck.resolve_decoder(d, device="cpu", dtype=F32)
    assert isinstance(m, HybridModel) and ck.decoder_family(d).name == "saritar"
    seq = C.toks(20, js["vocab"], 2)
    C.close(C.run_steps(C.engine(m), [[("a", seq)]])["a"], O.forward(js, w, seq))
    assert isinstance(ck.resolve_decoder("tiny", device="cpu"), LlamaModel)
    m = ck.resolve_decoder("saritar-tiny", device="cpu", dtype=F32, seed=3)
    assert isinstance(m, HybridModel) and m.cfg.name == "saritar-tiny"
    (tmp_path / "other").mkdir()
    (tmp_path / "other" / "config.json").write_text('{"architecture": "Unknown"}')
    with pytest.raises(NotImplementedError):
        ck.resolve_decoder(tmp_path / "other", device="cpu")
    cfg = json.loads((d / "config.json").read_text())
    cfg["vocab"] += 1
    (d / "config.json").write_text(json.dumps(cfg))
    with pytest.raises(ValueError, match="embed"):
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


def test_trace_replay_llama():
    """The same replay drives the Llama family: portions and decoded tokens agree with one pass."""
    from docqa_amd.engine.llm_engine import LLMEngine
    from docqa_amd.models.llama import LlamaConfig, LlamaModel

    m = LlamaModel(LlamaConfig.preset("tiny"), device="cpu", dtype=F32, seed=7)
    seq, other = C.toks(40, 4096, 1), C.toks(25, 4096, 2)

    def eng():
        return LLMEngine(m, max_batch=4, max_context=128, block_size=16, num_blocks=8, use_graphs=False, prefix_cache=False)

    one = C.run_steps(eng(), [[("a", seq)], [("b", other)]])
    two = C.run_steps(eng(), [[("a", seq[:20])], [("a", seq[20:21]), ("b", other[:9])], [("b", other[9:]), ("a", seq[21:])]])
    for k in one:
        C.close(two[k], one[k])


def test_qa_stack_over_saritar():
    """The RAG pipeline runs with a hybrid generator named by its preset."""
    from docqa_amd.pipeline.builder import StackConfig, build_stack

    pipe, _ = build_stack(StackConfig(llm="saritar-tiny", embed="tiny-bert", n_notes=20, max_batch=2, max_context=1024,
                                      use_graphs=False), device="cpu")
    pipe.answer("Which antibiotic was started?", C.SamplingParams(max_new_tokens=3, stop_on_eos=False))
    assert pipe.engine.state.num_free() == pipe.engine.state.slots
