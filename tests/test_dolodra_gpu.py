"""Dolodra on the HIP kernels, in fp32 and bf16, against the plain oracle."""
import sys
from pathlib import Path

import pytest
import torch

sys.path.insert(0, str(Path(__file__).parent))
import dolodra_cases as C  # noqa: E402

pytestmark = pytest.mark.gpu
DTYPES = [torch.float32, torch.bfloat16]


@pytest.fixture(autouse=True)
def _native():
    from docqa_amd import ops

    assert ops.load_native(), ops.native_error()
    torch.set_num_threads(4)


def test_stream_and_activations():
    C.elementwise_case("cuda")
    # odd shapes, then each GEMM with the activation in its epilogue
    C.gelu_linear_case("cuda", [(3, 40, 24), (1, 4096, 2048), (5, 12288, 512), (100, 12288, 512), (200, 14592, 256),
                                (600, 16384, 256)])
    C.rope_case("cuda")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("case", ["side_case", "norm_conv_case", "input_conv_case", "head_project_case", "latent_case", "latent_odd_case",
                                  "window_edge_case", "sink_case", "batch_latent_case"])
def test_mechanisms(case, dtype):
    getattr(C, case)("cuda", dtype)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(C.CONFIGS))
def test_models(name, dtype):
    if name in C.FP32_ONLY and dtype != torch.float32:
        pytest.skip("not a continuous function of its input")
    C.whole_case(name, "cuda", dtype)
    C.portions_case(name, "cuda", dtype)
    C.batch_case(name, "cuda", dtype)


@pytest.mark.parametrize("dtype", DTYPES)
def test_long_decode_and_far_tokens(dtype):
    C.long_decode_case("edge", "cuda", dtype)
    C.far_case("cuda", dtype)


@pytest.mark.parametrize("name", ["mixed", "odd"])
def test_generation(name):
    C.generate_case(name, "cuda")
    C.generate_case(name, "cuda", use_graphs=True)
    C.mixed_steps_case(name, "cuda")


def test_preemption_recomputes_state():
    C.preemption_case("mixed", "cuda")


@pytest.mark.parametrize("dtype", DTYPES)
def test_graph_replays_match_eager_steps(dtype):
    """A captured decode step replayed with eager work in between: the same tokens as eager
    steps, and capturing it leaves the convolution inputs alone."""
    js, w, m = C.make("mixed", "cuda", dtype, seed=40)
    prompts = [C.toks(n, js["vocab"], n) for n in (9, 30, 17)]
    sp = C.SamplingParams(max_new_tokens=25)
    eager = C.engine(m, tokens=512, slots=4).generate(prompts, sp)
    eng = C.engine(m, tokens=512, slots=4, use_graphs=True)
    for _ in range(3):
        assert eng.generate(prompts, sp) == eager
        torch.cuda.synchronize()
    assert any(g.graph is not None for g in eng._graphs.values())


def test_two_branch_steps_match(monkeypatch):
    """A captured step whose layers run mixer and feed-forward as two graph branches, replayed with
    eager work in between, gives the eager steps' tokens."""
    from docqa_amd.models import hybrid

    monkeypatch.setattr(hybrid, "FORK_MIN_BYTES", 0)
    js, w, m = C.make("mixed", "cuda", torch.bfloat16, seed=41)
    prompts = [C.toks(n, js["vocab"], n) for n in (9, 30, 17)]
    sp = C.SamplingParams(max_new_tokens=25)
    eager = C.engine(m, tokens=512, slots=4).generate(prompts, sp)
    eng = C.engine(m, tokens=512, slots=4, use_graphs=True)
    for _ in range(3):
        assert eng.generate(prompts, sp) == eager
        torch.cuda.synchronize()
    assert m._side_stream is not None


WIDE = C.conf(1024, 2048, [C.lat(16, 128, 64, 128, 512, 96, ff=4096), C.lat(32, 64, 64, 64, 512, 200, ff=2048, kv_from=0)],
              4, 256, 0.5, 30.0)


def test_narrow_products():
    """Few outputs of many rows (K split over bf16 slabs), and the short-K product behind the side
    gate at the row counts where its kernel changes."""
    from docqa_amd import ops

    g = torch.Generator().manual_seed(1)
    for M, N, K in ((600, 256, 512), (1024, 128, 4096), (2100, 256, 1024), (5000, 512, 256), (700, 64, 320)):
        x, w = torch.randn(M, K, generator=g), torch.randn(N, K, generator=g) * K ** -0.5
        P = ops.narrow_project(x.to("cuda", torch.bfloat16), w.to("cuda", torch.bfloat16))
        C.close(P.float().sum(0) if P.dim() == 3 else P, x.to(torch.bfloat16).float() @ w.to(torch.bfloat16).float().T,
                torch.bfloat16, (M, N, K))
    for M in (8, 9, 64, 65, 300):
        P, w = torch.randn(M, 64, generator=g), (torch.randn(256, 64, generator=g) / 8).to(torch.bfloat16)
        table, ids = torch.randn(9, 100, generator=g).to(torch.bfloat16), torch.randint(0, 9, (M,), generator=g, dtype=torch.int32)
        gate = C.O.gelu_tanh(P.to(torch.bfloat16).float()[:, :60]) * table[ids.long(), 40:].float()
        y = ops.side_project(P.to("cuda", torch.bfloat16), ids.cuda(), table.cuda(), 40, 60, w.cuda(), True)
        C.close(y, gate @ w[:, :60].float().T, torch.bfloat16, M)


@pytest.mark.parametrize("rows", [1, 3, 40, 200])
def test_wide_layers_take_the_gemm_plans(rows):
    """Sizes the split-K GEMM kernels accept: decode rows through the slab consumers agree with
    the same step on the reference operators."""
    from docqa_amd import ops
    from docqa_amd.models import dolodra
    from docqa_amd.models.hybrid import HybridModel

    m = HybridModel(dolodra.config_from_json(WIDE), device="cuda", seed=1)
    eng = C.engine(m, tokens=rows * 64, bs=64, slots=rows)
    ref = C.engine(m, tokens=rows * 64, bs=64, slots=rows)
    seqs = [C.toks(7, 2048, r) for r in range(rows)]
    steps = [[(str(r), s[:5]) for r, s in enumerate(seqs)], [(str(r), s[5:6]) for r, s in enumerate(seqs)],
             [(str(r), s[6:]) for r, s in enumerate(seqs)]]
    got = C.run_steps(eng, steps)
    if rows > 3:                       # the reference walks sequences one by one
        keep = [0, 1, rows - 1]
        steps = [[s for s in st if int(s[0]) in keep] for st in steps]
    with ops.use_reference():
        want = C.run_steps(ref, steps)
    for k in want:
        C.close(got[k], want[k].cpu(), torch.bfloat16, k)


@pytest.mark.parametrize("M", [300, 2500])
def test_long_prompt_prefill(M):
    """A prompt long enough for the prefill GEMMs: whole (keys and values of every head made), cut
    in portions, and the last tokens decoded (in the latent space)."""
    from docqa_amd.models import dolodra
    from docqa_amd.models.hybrid import HybridModel

    m = HybridModel(dolodra.config_from_json(WIDE), device="cuda", seed=2)
    seq = C.toks(M, 2048, 3)
    tail = [M - 1, M - 2, M // 2, 130, 1]

    def run(sizes):
        tr = C.TraceReplay(C.engine(m, tokens=4096, bs=64, slots=1))
        out, t = {}, 0
        for p in C.portions(seq, sizes):
            w = [q - t for q in tail if t <= q < t + len(p)]
            o = tr.step([{"id": "a", "tokens": p, "want": w}])
            for j, q in enumerate(w):
                out[q + t] = o[j]
            t += len(p)
        return torch.stack([out[q] for q in tail])

    whole = run([M])
    for sizes in ([100, 64, 2], [M - 2, 1, 1], [M // 2], [M - 66, 64, 2]):
        C.close(run(sizes), whole.cpu(), torch.bfloat16, sizes)
