"""Whole-model test bodies of a decoder family: ``ModelCases(configs, make, forward)`` with ``make(name,
device, dtype, seed)`` -> (config.json dict, weights, model) and ``forward`` the family's plain oracle."""
from __future__ import annotations

import torch

from docqa_amd.engine.llm_engine import SamplingParams
from docqa_amd.engine.scheduler import ContinuousEngine
from docqa_amd.engine.trace import TraceReplay
from saritar_cases import F32, close, engine, portions, run_steps, toks


class ModelCases:
    def __init__(self, make, forward):
        self.make, self.forward = make, forward

    def whole(self, name, device, dtype, T=45):
        js, w, m = self.make(name, device, dtype)
        seq = toks(T, js["vocab"], 1)
        res = []
        want = self.forward(js, w, seq, residuals=res)
        m.tap = []
        got = run_steps(engine(m), [[("a", seq)]])["a"]
        assert len(m.tap) == len(res) == len(js["layers"])
        for i, (a, b) in enumerate(zip(m.tap, res)):
            close(a, b, dtype, f"{name}: layer {i}")
        m.tap = None
        close(got, want, dtype, name)
        assert got.dtype == F32

    def portions(self, name, device, dtype, T=61, cuts=None):
        js, w, m = self.make(name, device, dtype, seed=2)
        seq = toks(T, js["vocab"], 3)
        want = self.forward(js, w, seq)
        for sizes in cuts or ([2] * (T // 2), [1] * T, [T - 8] + [1] * 8, [16, 16, 16], [15, 2, 17, 3, 1, 1, 9], [3, 1, 2, 31]):
            got = run_steps(engine(m), [[("a", p)] for p in portions(seq, sizes)])["a"]
            close(got, want, dtype, (name, sizes))

    def batch(self, name, device, dtype):
        """Requests of unequal length, portions beside decoded tokens, one left out for a while,
        pages and slots given back and taken again, against the oracle on each alone."""
        js, w, m = self.make(name, device, dtype, seed=4)
        eng = engine(m, tokens=160, bs=16, slots=3)
        V = js["vocab"]
        seqs = {"a": toks(50, V, 5), "b": toks(33, V, 6), "c": toks(9, V, 7), "d": toks(47, V, 8), "e": toks(1, V, 9)}
        want = {k: self.forward(js, w, s) for k, s in seqs.items()}
        at = dict.fromkeys(seqs, 0)
        got = {k: [] for k in seqs}
        tr = TraceReplay(eng)
        plan = [{"a": 20, "b": 1}, {"a": 1, "b": 2, "c": 5}, {"a": 1, "c": 1}, {"b": 16, "c": 1, "a": 1}, {"c": 2, "a": 13},
                {"b": 1, "a": 1, "d": 18}, {"b": 13, "d": 1}, {"d": 2, "a": 13, "e": 1}, {"d": 26}]
        for step in plan:
            es = [{"id": k, "tokens": seqs[k][at[k]:at[k] + n], "want": list(range(n))} for k, n in step.items()]
            out = tr.step(es)
            r = 0
            for k, n in step.items():
                got[k].append(out[r:r + n])
                r += n
                at[k] += n
                if at[k] == len(seqs[k]):
                    tr.finish(k)
        assert at == {k: len(s) for k, s in seqs.items()} and not tr.live
        assert eng.kv.allocator.num_free() == 10 and (eng.state is None or eng.state.num_free() == 3)
        for k in seqs:
            close(torch.cat(got[k]), want[k], dtype, (name, k))

    def long(self, name, device, dtype, T=150):
        """Long decoding, and a prompt of several chunks cut anywhere."""
        js, w, m = self.make(name, device, dtype, seed=6)
        seq = toks(T, js["vocab"], 10)
        want = self.forward(js, w, seq)
        for sizes in ([3] + [1] * (T - 3), [T], [64, 64], [63, 2, 66], [T - 20] + [1] * 20):
            close(run_steps(engine(m, bs=64), [[("a", p)] for p in portions(seq, sizes)])["a"], want, dtype, (name, sizes[:3]))

    # ------------------------------------------------------------------ generation
    def greedy(self, js, w, prompt, n):
        s = list(prompt)
        for _ in range(n):
            s.append(int(self.forward(js, w, s, F32)[-1].argmax()))
        return s[len(prompt):]

    def generate(self, name, device, use_graphs=False):
        """Greedy generation through the static engine and the continuous scheduler: chunked
        prefill, several batches, slots and blocks all given back."""
        js, w, m = self.make(name, device, F32, seed=20)
        prompts = [toks(n, js["vocab"], 30 + n) for n in (1, 5, 40, 19, 33)]
        sp = SamplingParams(max_new_tokens=7)
        want = [self.greedy(js, w, p, 7) for p in prompts]
        eng = engine(m, tokens=512, bs=16, slots=8, use_graphs=use_graphs, max_prefill_tokens=24)
        assert eng.generate(prompts, sp) == want
        assert eng.generate(prompts[:2], SamplingParams(max_new_tokens=7, temperature=0.9, top_k=1)) == want[:2]
        ce = ContinuousEngine(engine(m, tokens=512, bs=16, slots=3, use_graphs=use_graphs))
        assert ce.generate(prompts, sp) == want
        for e in (eng, ce.eng):
            assert e.kv.allocator.num_free() == 32 and (e.state is None or e.state.num_free() == e.state.slots)

    def mixed_steps(self, name, device):
        """Stall-free admission: prompt chunks ride in decode steps; the tokens do not change."""
        js, w, m = self.make(name, device, F32, seed=21)
        prompts = [toks(n, js["vocab"], 50 + n) for n in (4, 45, 20, 37)]
        ce = ContinuousEngine(engine(m, tokens=512, bs=16, slots=4))
        ce.mixed, ce.chunk_tokens = True, 16
        futs = [ce.submit(prompts[0], SamplingParams(max_new_tokens=12))]
        for _ in range(3):
            ce.step()
        futs += [ce.submit(p, SamplingParams(max_new_tokens=6)) for p in prompts[1:]]
        while not all(f.done() for f in futs):
            ce.step()
        assert ce.mixed_steps > 0
        for i, (f, p) in enumerate(zip(futs, prompts)):
            assert f.result() == self.greedy(js, w, p, 12 if i == 0 else 6)

    def preemption(self, name, device):
        """The pool runs dry mid-decode: the youngest request loses its blocks and its state slot
        and is computed again from its first token."""
        js, w, m = self.make(name, device, F32, seed=22)
        prompts = [toks(n, js["vocab"], 70 + n) for n in (15, 14, 13)]
        ce = ContinuousEngine(engine(m, tokens=64, bs=16, slots=3))
        ce.reserve_ahead = 1
        out = ce.generate(prompts, SamplingParams(max_new_tokens=20))
        assert ce.preempted > 0
        assert out == [self.greedy(js, w, p, 20) for p in prompts]
        assert ce.eng.kv.allocator.num_free() == 4

    def graphs(self, name, device, dtype):
        """A captured decode step replayed with eager work in between: the same tokens as eager
        steps, and capturing it leaves the states alone."""
        js, w, m = self.make(name, device, dtype, seed=40)
        prompts = [toks(n, js["vocab"], n) for n in (9, 30, 17)]
        sp = SamplingParams(max_new_tokens=25)
        eager = engine(m, tokens=512, slots=4).generate(prompts, sp)
        eng = engine(m, tokens=512, slots=4, use_graphs=True)
        for _ in range(3):
            assert eng.generate(prompts, sp) == eager
            torch.cuda.synchronize()
        assert any(g.graph is not None for g in eng._graphs.values())
