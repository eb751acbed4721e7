"""What every generator model shares: the LM head's greedy / sampling ends and the cache and
state a model declares to the engine.

A model lists the paged caches (:class:`~docqa_amd.engine.kv_cache.KVSpec`) and the recurrent
states (:class:`~docqa_amd.engine.kv_cache.StateSpec`) it needs; the engine allocates both,
hands out blocks and slots per request and passes what :meth:`Decoder.bind_caches` makes of
them to ``forward``.
"""
from __future__ import annotations

import torch

from .. import ops
from ..parallel import comm


class Decoder:
    # prompt-prefix reuse (block / token-granular KV caches) and the shared-prefix decode
    # kernels apply: everything a prompt leaves behind lives in its K/V blocks
    prefix_reuse = True
    # prefill always reads the paged cache (block tables / prefix lengths even at position 0)
    paged_prefill = False

    def kv_specs(self) -> list:
        raise NotImplementedError

    def state_specs(self) -> list:
        return []

    def bind_caches(self, kv, state) -> list:
        """Per-layer cache operands of ``forward`` from the engine's pools."""
        return kv.caches

    def activation_elems(self) -> int:
        """Peak activation elements per prefill token (KV pool sizing)."""
        raise NotImplementedError

    # ------------------------------------------------------------------ LM head
    def greedy_ids(self, x: torch.Tensor) -> torch.Tensor:
        """Greedy token ids int64 [R] of the final normed hidden rows ``x``: the LM-head GEMM
        with its argmax fused (mgemm.hip EPI_ARGMAX, no [R, vocab] logits) where the shape
        allows, the vocab-parallel pick resolved by one packed-key MAX all-reduce at TP > 1."""
        R = x.shape[0]
        N, K = self.lm_head.shape
        fused = ops.lm_head_argmax_ok(R, N, K) or (self.tp > 1 and 0 < R <= ops.MID_M_MAX
                                                   and ops.lm_head_argmax_shape_ok(N, K))
        fused = fused and not (x.is_cuda and x.dtype != torch.bfloat16)
        if self.tp == 1:
            if fused:
                return ops.lm_head_argmax(x, self.lm_head, self.cfg.vocab_size)
            return self.greedy(ops.lm_head_logits(x, self.lm_head))
        if fused and self.vocab_valid > 0:
            ids, vals = ops.lm_head_argmax(x, self.lm_head, self.vocab_valid, with_values=True)
        else:
            logits = ops.lm_head_logits(x, self.lm_head)[:, : max(1, self.vocab_valid)]
            ids = ops.argmax(logits)
            vals = logits.gather(1, ids[:, None])[:, 0].float()
        if self.vocab_valid == 0:
            vals = torch.full_like(vals, float("-inf"))
        return comm.tp_argmax(vals, ids + self.vocab_start)

    def greedy(self, logits: torch.Tensor) -> torch.Tensor:
        """argmax over the (possibly vocab-parallel) logits -> int64 [R]."""
        if self.tp == 1:
            return ops.argmax(logits)
        valid = logits[:, : max(1, self.vocab_valid)]
        idx = ops.argmax(valid)
        val = valid.gather(1, idx[:, None])[:, 0].float()
        if self.vocab_valid == 0:
            val = torch.full_like(val, float("-inf"))
        return comm.tp_argmax(val, idx + self.vocab_start)

    def full_logits(self, logits: torch.Tensor) -> torch.Tensor:
        full = comm.tp_all_gather_last(logits)
        return full[:, : self.cfg.vocab_size]
