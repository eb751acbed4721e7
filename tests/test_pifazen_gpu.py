"""Pifazen on the HIP kernels, in fp32 and bf16, against the plain oracle."""
import sys
from pathlib import Path

import pytest
import torch

sys.path.insert(0, str(Path(__file__).parent))
import pifazen_cases as C  # noqa: E402
from test_pifazen_cpu import MECHANISMS  # noqa: E402

pytestmark = pytest.mark.gpu
F32, BF16 = torch.float32, torch.bfloat16
DTYPES = [F32, BF16]


@pytest.fixture(autouse=True)
def _native():
    from docqa_amd import ops

    assert ops.load_native(), ops.native_error()
    torch.set_num_threads(4)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("case", MECHANISMS)
def test_mechanisms(case, dtype):
    getattr(C, case)("cuda", dtype)


# (the norm of one element is its sign, which rounding decides near zero: "ones" runs in fp32)
@pytest.mark.parametrize("name,dtype", [(n, d) for n in C.CONFIGS for d in DTYPES if (n, d) != ("ones", BF16)])
def test_models(name, dtype):
    C.MODELS.whole(name, "cuda", dtype)
    C.MODELS.portions(name, "cuda", dtype)
    C.MODELS.batch(name, "cuda", dtype)


@pytest.mark.parametrize("dtype", DTYPES)
def test_long_decoding(dtype):
    C.MODELS.long("edge", "cuda", dtype)


@pytest.mark.parametrize("name", ["mixed", "odd"])
def test_generation(name):
    C.MODELS.generate(name, "cuda")
    C.MODELS.generate(name, "cuda", use_graphs=True)
    C.MODELS.mixed_steps(name, "cuda")


def test_preemption_recomputes_state():
    C.MODELS.preemption("mixed", "cuda")


@pytest.mark.parametrize("dtype", DTYPES)
def test_graph_replays_match_eager_steps(dtype):
    C.MODELS.graphs("mixed", "cuda", dtype)


# widths that the GEMM kernels, the packed attention and the grouped tiles accept
_WD = C.delta(8, 8, 128, 128, 4, C.moe(8, 4, 3, 256, 4, 2, 2.0, 7.0))
WIDE = C.conf(1024, 2048, [_WD, C.lat(8, 128, 64, 128, 512, 768, base=5e5, mlp=C.dense(2048)), C.again(_WD, 0),
                           C.lat2(8, 128, 64, 128, 512, (8.0, 256.0, 32.0, 1.0), base=1e6, mlp=C.moe(4, 2, 2, 512, 2, 1, 1.5, 7.0))])


def wide_model(seed):
    js = WIDE
    w = C.O.random_weights(js, seed, rank=(64, 128))
    C.settle_routing(w, js)
    return C.HybridModel(C.pifazen.config_from_json(js), device="cuda", weights=w)


@pytest.mark.parametrize("rows", [1, 3, 40, 300])
def test_wide_layers_take_the_gemm_plans(rows):
    """Decode rows through the slab consumers and the experts' kernels of either kind agree with the same
    step on the reference operators."""
    from docqa_amd import ops

    m = wide_model(1)
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
        C.close(got[k], want[k].cpu(), BF16, k)


@pytest.mark.parametrize("M", [300, 2500])
def test_long_prompt_prefill(M):
    """A prompt long enough for the prefill GEMMs and the sorted experts: whole, cut in portions, and the
    last tokens decoded."""
    from docqa_amd.engine.trace import TraceReplay

    m = wide_model(2)
    seq = C.toks(M, 2048, 3)
    tail = [M - 1, M - 2, M // 2, 130, 1]

    def run(sizes):
        tr = TraceReplay(C.engine(m, tokens=4096, bs=64, slots=1))
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
        C.close(run(sizes), whole.cpu(), BF16, sizes)
