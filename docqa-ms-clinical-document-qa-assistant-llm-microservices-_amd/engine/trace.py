"""Replay of a request trace: given token ids are fed step by step through the engine's own
prefill / decode forwards, block allocator and state pool, and logits are written out.
Nothing is sampled.

A step is a JSON object ``{"step": n, "entries": [{"id", "tokens", "want"}], "end": [ids]}``:
each entry's next tokens of a request (admitted at its first entry), ``want`` the places
among them whose logits are asked for, ``end`` the requests that finish after the step.  All
entries of a step are one batch, as in a continuous-batching step: requests that bring one
more token are decode rows, the others prompt portions beside them (``forward_mixed``).
"""
from __future__ import annotations

import json
from dataclasses import dataclass, field
from pathlib import Path

import torch

from .llm_engine import LLMEngine


@dataclass
class _Live:
    tokens: list = field(default_factory=list)
    blocks: list = field(default_factory=list)
    slots: list = field(default_factory=list)


class TraceReplay:
    def __init__(self, engine: LLMEngine):
        self.eng = engine
        self.live: dict[str, _Live] = {}

    def _admit(self, rid: str) -> _Live:
        r = self.live.get(rid)
        if r is None:
            if len(self.live) >= self.eng.max_batch:
                raise MemoryError(f"more than {self.eng.max_batch} live requests")
            r = self.live[rid] = _Live(slots=self.eng.state.alloc(1) if self.eng.state is not None else [])
        return r

    def finish(self, rid: str) -> None:
        r = self.live.pop(rid)
        self.eng.kv.allocator.free(r.blocks)
        if r.slots:
            self.eng.state.free(r.slots)

    @torch.inference_mode()
    def step(self, entries: list[dict]) -> torch.Tensor | None:
        """One batch; logits fp32 [wanted, vocab] in the order of the entries and their
        ``want``, or None when nothing is wanted."""
        eng = self.eng
        dec, pre = [], []                       # (entry index, request, first position)
        for i, e in enumerate(entries):
            if not e["tokens"]:
                continue
            r = self._admit(e["id"])
            start = len(r.tokens)
            r.tokens += [int(t) for t in e["tokens"]]
            if len(r.tokens) > eng.max_context:
                raise ValueError(f"request {e['id']}: {len(r.tokens)} tokens exceed the context {eng.max_context}")
            need = eng.kv.blocks_for(len(r.tokens)) - len(r.blocks)
            if need > 0:
                r.blocks += eng._retry(lambda: eng.kv.allocator.alloc(need))
            (dec if start > 0 and len(e["tokens"]) == 1 else pre).append((i, r, start))
        if not dec and not pre:
            return None
        n, g, dmeta, pmeta = len(dec), None, None, None
        if dec:
            g = eng._get_graph(n, greedy=False)
            eng.load_rows(g, [r.tokens[-1] for _, r, _ in dec], [s for _, _, s in dec], [r.blocks for _, r, _ in dec],
                          [s for _, r, _ in dec for s in r.slots])
            dmeta = eng._decode_meta(g)
        if pre:
            ids, pmeta, cu = eng.prefill_batch([r.tokens for _, r, _ in pre], [r.blocks for _, r, _ in pre],
                                               [s for _, _, s in pre], [s for _, r, _ in pre for s in r.slots])
            if pmeta.block_tables is None and dec:
                eng.page_prefill(pmeta, [r.blocks for _, r, _ in pre], [s for _, _, s in pre])
        first = {i: k for k, (i, _, _) in enumerate(dec)}
        first.update({i: n + int(cu[k]) for k, (i, _, _) in enumerate(pre)})
        rows = [first[i] + w for i, e in enumerate(entries) for w in e.get("want", [])]
        # (nothing wanted: the last row's logits are computed and dropped)
        index = torch.tensor(rows or [n + int(cu[-1]) - 1 if pre else n - 1], dtype=torch.long, device=eng.device)
        model = eng.model
        if not pre:
            out = model.forward(g.tokens, dmeta, eng.caches, logits_index=index)
        elif not dec:
            out = model.forward(ids, pmeta, eng.caches, logits_index=index)
        else:
            out = model.forward_mixed(torch.cat([g.tokens, ids]), n, dmeta, pmeta, eng.caches, index,
                                      return_logits=True)
        return model.full_logits(out).float() if rows else None


def replay(engine: LLMEngine, lines, out_dir: Path, done=print) -> None:
    """Run every step of ``lines``: ``out_dir/<step>.f32`` (little-endian fp32 [wanted, vocab])
    where logits are wanted, then ``done("done <step>")``."""
    tr = TraceReplay(engine)
    for line in lines:
        if not line.strip():
            continue
        st = json.loads(line)
        logits = tr.step(st.get("entries", []))
        if logits is not None:
            (out_dir / f"{st['step']}.f32").write_bytes(logits.cpu().numpy().astype("<f4").tobytes())
        elif engine.device.type == "cuda":
            torch.cuda.synchronize()
        for rid in st.get("end", []):
            tr.finish(rid)
        done(f"done {st['step']}")


def main(argv: list[str] | None = None) -> int:
    import argparse
    import sys

    ap = argparse.ArgumentParser(prog="trace_run", description="Replay a request trace (JSON steps on standard input) "
                                 "through the engine and write logits.")
    ap.add_argument("--model", required=True, help="checkpoint directory (config.json + model.safetensors)")
    ap.add_argument("--dtype", choices=("bfloat16", "float32"), default="bfloat16")
    ap.add_argument("--out", required=True, help="directory the logits are written to")
    ap.add_argument("--max-tokens", type=int, required=True,
                    help="most tokens live requests hold together, each rounded up to whole cache blocks")
    ap.add_argument("--max-requests", type=int, default=4, help="most live requests (state slots)")
    ap.add_argument("--device", default="cuda", help="cuda (MI355X) | cpu (reference operators)")
    a = ap.parse_args(argv)

    from .. import ops
    from ..models import checkpoint as ck

    dtype = getattr(torch, a.dtype)
    if a.device != "cpu":
        if dtype not in ck.decoder_family(a.model).gpu_dtypes:
            print(f"{a.model}: its kernels do not run in {a.dtype}", file=sys.stderr)
            return 3
        if not torch.cuda.is_available():
            print("no GPU (--device cpu runs the reference operators)", file=sys.stderr)
            return 1
        if not ops.load_native(build_if_missing=True):
            raise RuntimeError(ops.native_error())
    torch.backends.cuda.matmul.allow_tf32 = False
    bs = 64
    blocks = max(1, a.max_tokens // bs)
    model = ck.resolve_decoder(a.model, device=a.device, dtype=dtype)
    eng = LLMEngine(model, max_batch=a.max_requests, max_context=blocks * bs, block_size=bs, num_blocks=blocks,
                    use_graphs=False, prefix_cache=False, state_slots=a.max_requests)
    out = Path(a.out)
    out.mkdir(parents=True, exist_ok=True)
    replay(eng, sys.stdin, out, done=lambda s: print(s, flush=True))
    return 0
