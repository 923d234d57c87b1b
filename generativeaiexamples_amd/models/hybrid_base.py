"""What the hybrid decoders share towards the serving engine: state-slot bookkeeping, the per-step (cu, slot, ctx, page
table) rows, the static inputs of captured decode graphs and checkpoint loading; the execution order of a looped block
and the packed weights of gated experts.

A model class supplies ``load_state`` (checkpoint tensors -> device weights in ``self.w``), ``_alloc_state`` (registers
its recurrent states in ``self.pool``), ``kv_layout`` and ``forward``. A decoder whose layers are all attention sets
``has_recurrent_state = False``: it takes no state slots, and cached prefixes can be reused.
"""
from __future__ import annotations

import os
from typing import Dict, List, Tuple

import torch

from .. import ops
from ..engine.state_pool import StatePool
from .common import ForwardBatch


def loop_runs(n_layers: int, start: int, stop: int, times: int) -> List[Tuple[int, int]]:
    """Execution order as (layer, pass) pairs: layers start .. stop-1 run `times` times in a row (0: no looped block), the
    others once."""
    if not times:
        return [(i, 0) for i in range(n_layers)]
    return ([(i, 0) for i in range(start)] + [(i, t) for t in range(times) for i in range(start, stop)] +
            [(i, 0) for i in range(stop, n_layers)])


def pad_rows(t: torch.Tensor, n: int) -> torch.Tensor:
    """fp32 rows of t followed by zero rows up to a multiple of n (the matrix-core GEMMs' column grid)."""
    return torch.cat([t.float(), torch.zeros((-t.shape[0]) % n, *t.shape[1:])])


def stack_gated_experts(sd: Dict[str, torch.Tensor], p: str, n_experts: int, grid: int) -> Tuple[torch.Tensor, torch.Tensor]:
    """Expert tensors `<p>e<j>.gate / .up / .down` -> (gate_up [E, 2 F', D] with gate / up rows interleaved per 16, down
    [E, D, F']), fp32; F' = the experts' width padded with zeros to `grid` (a zero gate / up row contributes nothing)."""
    gu, dn = [], []
    for j in range(n_experts):
        q = f"{p}e{j}."
        gu.append(ops.interleave_gate_up(pad_rows(sd[q + "gate"], grid), pad_rows(sd[q + "up"], grid)))
        dn.append(pad_rows(sd[q + "down"].t(), grid).t())
    return torch.stack(gu), torch.stack(dn)


class HybridDecoderBase:
    has_recurrent_state = True       # no prefix-cache reuse: a cached prefix has no recurrent state to resume from
    attention_backend = "window"     # the paged window attention kernels: no flash-attention tile lists

    w: Dict[str, torch.Tensor]
    pool: StatePool
    device: torch.device

    def load_hf_state(self, sd: Dict[str, torch.Tensor]):
        return self.load_state(sd)

    def load_safetensors_dir(self, path: str):
        from safetensors.torch import load_file

        sd = {}
        for f in sorted(os.listdir(path)):
            if f.endswith(".safetensors"):
                sd.update(load_file(os.path.join(path, f)))
        return self.load_state(sd)

    def num_params(self) -> int:
        return sum(t.numel() for t in self.w.values())

    def set_state_slots(self, n: int):
        """Engine hook: size the state pool for n live sequences (before any request is admitted)."""
        if self.has_recurrent_state and n != self.pool.n_slots:
            self.pool = StatePool(n, self.device)
            if self.w:
                self._alloc_state()

    def release_request(self, sid: int):
        if self.has_recurrent_state:
            self.pool.release(sid)

    def prepare_batch(self, fb: ForwardBatch):
        """Engine hook: one (cu, slot, ctx, page table) row per sequence of the step - prompt portions first, then
        single decoded tokens - and fresh state for sequences that start at position 0."""
        P = len(fb.prefill_qlen)
        nd = fb.num_tokens - fb.num_prefill_tokens
        pctx = fb.prefill_ctx_host or []
        dctx = fb.decode_ctx_host or []
        sids = (fb.seq_ids or []) if self.has_recurrent_state else []
        slots = [self.pool.slot(sid, pctx[i] == fb.prefill_qlen[i]) for i, sid in enumerate(sids[:P])]
        slots += [self.pool.slot(sid, dctx[j] == 1 if j < len(dctx) else False) for j, sid in enumerate(sids[P:])]
        cu = [0]
        for n in fb.prefill_qlen:
            cu.append(cu[-1] + n)
        cu += [cu[-1] + j + 1 for j in range(nd)]
        dev = self.device
        extra = dict(cu=torch.tensor(cu, dtype=torch.int32).to(dev, non_blocking=True))
        if self.has_recurrent_state:
            extra["slots"] = torch.tensor(slots, dtype=torch.int32).to(dev, non_blocking=True)
        parts_c = [t for t in (fb.prefill_ctx if P else None, fb.decode_ctx if nd else None) if t is not None]
        parts_b = [t for t in (fb.prefill_block_tables if P else None, fb.decode_block_tables if nd else None)
                   if t is not None]
        extra["ctx"] = parts_c[0] if len(parts_c) == 1 else torch.cat(parts_c)
        extra["bt"] = parts_b[0] if len(parts_b) == 1 else torch.cat(parts_b)
        fb.extra = extra

    def graph_static_inputs(self, bs: int) -> dict:
        """Static inputs of a captured decode graph of bs rows (the engine's ctx / page-table tensors complete them)."""
        i32 = dict(dtype=torch.int32, device=self.device)
        out = dict(cu=torch.arange(bs + 1, **i32))
        if self.has_recurrent_state:
            out["slots"] = torch.full((bs,), self.pool.pad_slot, **i32)
        return out

    def fill_graph_inputs(self, extra: dict, seq_ids, n: int):
        if not self.has_recurrent_state:
            return
        ids = torch.tensor([self.pool.slot(s, False) for s in seq_ids] +
                           [self.pool.pad_slot] * (extra["slots"].numel() - n), dtype=torch.int32)
        extra["slots"].copy_(ids, non_blocking=True)
