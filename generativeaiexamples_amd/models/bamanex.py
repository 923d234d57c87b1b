"""Bamanex: a decoder of parallel layers - attention and feed-forward read the same stream, each through its own norm -
with sliding-window attention over unit-norm queries and keys, dense or mixture-of-experts feed-forwards and a looped
block of layers.

Architecture (every size and constant comes from ``config.json``):
  * token embedding; ``x += ls1 * attention(N1(x)) + ls2 * ff(N2(x))`` with per-channel layer scales and zero-centred
    RMS-norm weights (``x / rms(x) * (1 + w)``); a layer may have no feed-forward; the head is its own matrix and the
    logits are multiplied by ``logit_scale``;
  * ``loop``: layers ``start .. stop-1`` run ``times`` times with the same weights, each pass with its own KV cache;
  * attention: GQA with biases on all four projections; the first ``rot.dims`` channels of every q and k head rotated in
    the rotate-half layout with Llama-3.1 frequency scaling, then q and k divided by their root mean square per head; sliding
    window ``0 <= i - j < mask.size``; a learned value-less sink score per head in the softmax denominator; every head's
    output times ``sigmoid(W_g h)``, one number per head;
  * feed-forward ``dense``: ``W_down (gelu_tanh(W_gate h) * (W_up h))``; ``moe``: softmax router scores, the ``top`` largest
    renormalised, over experts ``W_down (g sigmoid(1.702 g) (u + 1))`` with ``g = min(W_gate h, limit)``,
    ``u = clamp(W_up h, +-limit)``, plus a shared expert of that form times ``sigmoid(w_sg . h)``.

MI355X mapping. The residual stream, norms, positions and angles, attention scores and weights and the router are fp32;
projections run in the model dtype (bf16 MFMA GEMMs with fp32 accumulation, or true fp32). One kernel between two layers
adds both scaled branch outputs and writes both norms of the new sum. q | k | v | head gates are one GEMM; rotation, unit
norm and cache write are one kernel; the attention kernel applies sink and head gate. K / V pages come from the engine's
paged cache, one cache layer per attention run; nothing else is carried from step to step, so there are no state slots and
cached prefixes are reusable. A step's rows - prompt portions and single decoded tokens alike - are addressed by
device-side (cu, ctx, page table) vectors, so pure-decode steps replay a captured HIP graph.
"""
from __future__ import annotations

import json
import os
from dataclasses import dataclass
from typing import Dict, List, Optional, Tuple

import torch

from .. import ops
from ..engine.state_pool import StatePool
from ..parallel.dist import DistContext, get_context
from .common import ForwardBatch
from .hybrid_base import HybridDecoderBase, loop_runs, pad_rows, stack_gated_experts

MIXERS = ("attention",)
ROUTE_EPS = 1e-20               # added to the sum of the chosen router scores


@dataclass
class BamanexConfig:
    vocab_size: int
    hidden_size: int
    layers: Tuple[dict, ...]                 # {"type", "mixer": {...}, "mlp": {"kind": "dense" | "moe", ...} | None}
    loop_start: int = 0
    loop_stop: int = 0
    loop_times: int = 0                      # 0: no looped block
    rms_eps: float = 1e-6
    logit_scale: float = 1.0
    name: str = "bamanex"
    max_position: int = 1 << 20              # angles are computed from the position: no table to outgrow
    bos_token_id: Optional[int] = None
    eos_token_ids: Tuple[int, ...] = ()

    def __post_init__(self):
        layers = []
        for i, l in enumerate(self.layers):
            if l["type"] not in MIXERS:
                raise ValueError(f"layer {i}: unknown mixer type {l['type']!r}")
            m = dict(l["mixer"])
            m.setdefault("kv_heads", m["heads"])
            m.setdefault("vdim", m["dim"])
            m.setdefault("scale", m["dim"] ** -0.5)
            m["window"] = int((m.get("mask") or {}).get("size") or 0)   # 0: every earlier position
            if m["heads"] % m["kv_heads"]:
                raise ValueError(f"layer {i}: heads must be a multiple of kv_heads")
            rot = dict(m.get("rot") or {})
            dims = rot["dims"] = int(rot.get("dims") or 0)
            rot.setdefault("base", 10000.0)
            if dims % 2 or not 0 <= dims <= m["dim"]:
                raise ValueError(f"layer {i}: the rotation covers an even number of a head's channels")
            m["rot"] = rot
            ml = l.get("mlp")
            if ml is not None:
                ml = dict(ml)
                kind = ml.setdefault("kind", "dense")
                if kind not in ("dense", "moe"):
                    raise ValueError(f"layer {i}: unknown feed-forward kind {kind!r}")
                if kind == "moe" and not 1 <= ml["router"]["top"] <= min(16, ml["router"]["experts"]):
                    raise ValueError(f"layer {i}: 1 <= top <= min(16, experts)")
            layers.append(dict(l, mixer=m, mlp=ml))
        self.layers = tuple(layers)
        if self.loop_times and not (0 <= self.loop_start < self.loop_stop <= len(self.layers)):
            raise ValueError("loop: need 0 <= start < stop <= number of layers")

    @property
    def num_layers(self) -> int:
        return len(self.layers)

    @property
    def head_dim(self) -> int:  # engine sizing hooks: the widest cached key row
        return max([l["mixer"]["dim"] for l in self.layers] or [16])

    def runs(self) -> List[Tuple[int, int]]:
        """Execution order as (layer, pass) pairs; a looped layer appears once per pass."""
        return loop_runs(len(self.layers), self.loop_start, self.loop_stop, self.loop_times)

    @staticmethod
    def from_json(path_or_dict) -> "BamanexConfig":
        if isinstance(path_or_dict, dict):
            c, name = path_or_dict, "bamanex"
        else:
            with open(os.path.join(path_or_dict, "config.json")) as f:
                c = json.load(f)
            name = os.path.basename(os.path.normpath(path_or_dict)) or "bamanex"
        lp = c.get("loop") or {}
        eos = c.get("eos_token_id", ())
        return BamanexConfig(
            vocab_size=int(c["vocab"]), hidden_size=int(c["width"]), layers=tuple(c["layers"]),
            loop_start=int(lp.get("start", 0)), loop_stop=int(lp.get("stop", 0)), loop_times=int(lp.get("times", 0)),
            rms_eps=float((c.get("norm") or {}).get("eps", 1e-6)), logit_scale=float(c.get("logit_scale", 1.0)),
            name=c.get("name", name), max_position=int(c.get("max_position", 1 << 20)),
            bos_token_id=c.get("bos_token_id"), eos_token_ids=tuple(eos) if isinstance(eos, (list, tuple)) else (eos,))

    @staticmethod
    def tiny(**kw) -> "BamanexConfig":
        att = dict(heads=4, kv_heads=2, dim=16, vdim=24, scale=0.4, mask=dict(size=20),
                   rot=dict(base=1000.0, dims=8, scaling=dict(factor=4.0, low=1.0, high=4.0, original=64)))
        dense = dict(kind="dense", ff=96)
        moe = dict(kind="moe", expert=dict(ff=32, limit=2.0), shared=dict(ff=48, limit=3.0), router=dict(experts=6, top=2))
        base = dict(vocab_size=512, hidden_size=64, name="tiny-bamanex", rms_eps=1e-5, logit_scale=0.8, loop_start=1,
                    loop_stop=3, loop_times=2,
                    layers=(dict(type="attention", mixer=att, mlp=dense), dict(type="attention", mixer=att, mlp=moe),
                            dict(type="attention", mixer=att, mlp=None), dict(type="attention", mixer=att, mlp=moe)))
        base.update(kw)
        return BamanexConfig(**base)

    @staticmethod
    def sized(width: int, n_layers: int, ff: int, heads: int, head_dim: int, window: int = 1024, vocab: int = 32768,
              experts: int = 8, top: int = 2, moe_every: int = 2, **kw) -> "BamanexConfig":
        """A regular stack for benchmarks: every `moe_every`-th layer (0: none) carries `experts` experts of ff / top (the
        active routed feed-forward equals a dense ff) plus a shared expert of ff / 4, the others a dense ff."""
        att = dict(heads=heads, kv_heads=max(1, heads // 4), dim=head_dim, vdim=head_dim, scale=head_dim ** -0.5,
                   mask=dict(size=window),
                   rot=dict(base=500000.0, dims=head_dim // 2,
                            scaling=dict(factor=8.0, low=1.0, high=4.0, original=8192)))
        dense = dict(kind="dense", ff=ff)
        moe = dict(kind="moe", expert=dict(ff=ff // top, limit=7.0), shared=dict(ff=ff // 4, limit=7.0),
                   router=dict(experts=experts, top=top))
        layers = tuple(dict(type="attention", mixer=att, mlp=moe if moe_every and (i + 1) % moe_every == 0 else dense)
                       for i in range(n_layers))
        base = dict(vocab_size=vocab, hidden_size=width, layers=layers, name=f"bamanex-{width}x{n_layers}")
        base.update(kw)
        return BamanexConfig(**base)


def random_state(cfg: BamanexConfig, seed: int = 0) -> Dict[str, torch.Tensor]:
    """A random checkpoint (tensor names and shapes of the safetensors layout, fp32 values) with magnitudes that keep
    activations and scores in a trained model's range."""
    g = torch.Generator().manual_seed(seed)
    D = cfg.hidden_size
    rn = lambda *s, std=1.0: torch.randn(*s, generator=g) * std  # noqa: E731
    lin = lambda o, i: rn(o, i, std=i ** -0.5)  # noqa: E731
    sd: Dict[str, torch.Tensor] = {"embed": rn(cfg.vocab_size, D), "head": lin(cfg.vocab_size, D) * 2.0,
                                   "final.norm": rn(D, std=0.1)}

    def gated(p, F_):
        sd[p + "gate"], sd[p + "up"], sd[p + "down"] = lin(F_, D) * 1.5, lin(F_, D) * 1.5, lin(D, F_)

    for i, l in enumerate(cfg.layers):
        p, x, m = f"l{i}.", f"l{i}.mix.", l["mixer"]
        H, G, dk, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        sd[p + "norm1"], sd[p + "ls1"] = rn(D, std=0.1), 0.5 + rn(D, std=0.1)
        for n, rows in (("q", H * dk), ("k", G * dk), ("v", G * dv)):
            sd[x + n], sd[x + n + ".b"] = lin(rows, D), rn(rows, std=0.1)
        sd[x + "sink"], sd[x + "g"] = rn(H), lin(H, D)
        sd[x + "o"], sd[x + "o.b"] = lin(D, H * dv), rn(D, std=0.1)
        ml = l["mlp"]
        if ml is None:
            continue
        sd[p + "norm2"], sd[p + "ls2"] = rn(D, std=0.1), 0.5 + rn(D, std=0.1)
        if ml["kind"] == "dense":
            gated(p + "mlp.", ml["ff"])
            continue
        for e in range(ml["router"]["experts"]):
            gated(p + f"mlp.e{e}.", ml["expert"]["ff"])
        sd[p + "mlp.router"] = lin(ml["router"]["experts"], D) * 2.0
        if ml.get("shared"):
            gated(p + "mlp.shared.", ml["shared"]["ff"])
            sd[p + "mlp.shared.sg"] = lin(1, D)
    return sd


class BamanexModel(HybridDecoderBase):
    """Weights (plain tensors) + forward for the serving engine (the hooks of LlamaModel / PinavikModel)."""

    has_recurrent_state = False      # everything a step leaves behind is in the KV pages

    def __init__(self, cfg: BamanexConfig, device=None, dtype=torch.bfloat16, dist_ctx: DistContext | None = None):
        self.cfg = cfg
        self.ctx = dist_ctx or get_context()
        assert self.ctx.tp_size == 1, "Bamanex runs TP=1"
        self.device = torch.device(device) if device is not None else self.ctx.device
        self.dtype = dtype
        self.runs = cfg.runs()
        self.kv_index = {r: j for j, r in enumerate(self.runs)}
        self.num_kv_layers = len(self.runs)
        self.hq = max([l["mixer"]["heads"] for l in cfg.layers] or [1])
        self.hkv = max([l["mixer"]["kv_heads"] for l in cfg.layers] or [1])
        self.vocab_local, self.vstart = cfg.vocab_size, 0
        self.lora_names: list = []
        self.w: Dict[str, torch.Tensor] = {}
        self.pool = StatePool(0, self.device)          # no recurrent layers: stays empty
        self.capture_residuals: Optional[list] = None  # numerics debugging: the residual stream after every layer run

    # ------------------------------------------------------------------ engine sizing hooks
    def kv_layout(self) -> List[Tuple[int, int, int]]:
        """(kv heads, key size, value size) of every paged cache layer: one per layer run."""
        ms = [self.cfg.layers[i]["mixer"] for i, _t in self.runs]
        return [(m["kv_heads"], m["dim"], m["vdim"]) for m in ms]

    # ------------------------------------------------------------------ weights
    def load_state(self, sd: Dict[str, torch.Tensor]):
        """Checkpoint tensors (the safetensors names) -> device weights: projections in the model dtype, per-channel
        tables fp32, same-input projections fused, norm weights stored as 1 + w (the final one times the logit scale),
        expert matrices stacked with gate / up rows interleaved per 16 (zero rows up to the GEMMs' grids: a zero gate / up
        row contributes nothing)."""
        c, dev, dt = self.cfg, self.device, self.dtype
        f32 = lambda t: t.to(torch.float32).to(dev).contiguous()  # noqa: E731
        mat = lambda t: t.to(torch.float32).to(dev, dt).contiguous()  # noqa: E731
        bf = dt == torch.bfloat16
        w = self.w = {}
        w["embed"], w["head"] = mat(sd["embed"]), mat(pad_rows(sd["head"], 16))   # padded logits are cut off by forward()
        w["final.norm"] = f32((1 + sd["final.norm"].float()) * c.logit_scale)

        def gated(src, dst, fused, extra=()):
            # wide feed-forwards padded with zeros to the split-K decode GEMM's grid; fused: rows interleaved for the gated
            # epilogue of the GEMM
            wide = 512 if bf and sd[src + "gate"].shape[0] >= 1024 else 16
            gate, up = pad_rows(sd[src + "gate"], wide), pad_rows(sd[src + "up"], wide)
            rows = torch.cat([gate, up] + [sd[e].float().reshape(1, -1) for e in extra])
            w[dst + "in"] = mat(ops.interleave_gate_up(gate, up) if fused else pad_rows(rows, 16))
            w[dst + "down"] = mat(pad_rows(sd[src + "down"].t(), wide).t())

        for i, l in enumerate(c.layers):
            p, x, m = f"l{i}.", f"l{i}.mix.", l["mixer"]
            w[p + "norm1"], w[p + "ls1"] = f32(1 + sd[p + "norm1"].float()), f32(sd[p + "ls1"])
            w[x + "in"] = mat(pad_rows(torch.cat([sd[x + k].float() for k in "qkvg"]), 16))
            bias = torch.cat([sd[x + k + ".b"].float() for k in "qkv"])
            w[x + "in.b"] = mat(torch.cat([bias, torch.zeros(w[x + "in"].shape[0] - bias.numel())]))
            w[x + "o"], w[x + "o.b"], w[x + "sink"] = mat(sd[x + "o"]), mat(sd[x + "o.b"]), f32(sd[x + "sink"])
            w[x + "inv_freq"] = ops.rope_inv_freq(m["rot"]["dims"], m["rot"]["base"], m["rot"].get("scaling")).to(dev)
            ml, q = l["mlp"], p + "mlp."
            if ml is None:
                continue
            w[p + "norm2"], w[p + "ls2"] = f32(1 + sd[p + "norm2"].float()), f32(sd[p + "ls2"])
            if ml["kind"] == "dense":
                gated(q, q, bf)
                continue
            w[q + "router"] = mat(pad_rows(sd[q + "router"], 16))
            gate_up, down = stack_gated_experts(sd, q, ml["router"]["experts"], 64 if bf else 16)
            w[q + "gate_up"], w[q + "e.down"] = mat(gate_up), mat(down)
            if ml.get("shared"):
                gated(q + "shared.", q + "shared.", False, (q + "shared.sg",))
        return self

    def random_init(self, seed: int = 0):
        return self.load_state(random_state(self.cfg, seed))

    # ------------------------------------------------------------------ branches
    def _attention(self, h, i, run, fb, kv, seq):
        m, w, x = self.cfg.layers[i]["mixer"], self.w, f"l{i}.mix."
        H, G, dk, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        proj = ops.linear(h, w[x + "in"], w[x + "in.b"])
        a, b = H * dk, (H + G) * dk
        c = b + G * dv
        kc, vc = kv.layer(self.kv_index[run])
        q = ops.rotary_half_kv_write(proj[:, :a], proj[:, a:b], proj[:, b:c], fb.positions, fb.slots, kc, vc, H, G, dk, dv,
                                     w[x + "inv_freq"], self.cfg.rms_eps)
        att = ops.window_attention(q, kc, vc, seq["bt"], seq["cu"], seq["ctx"], H, G, dk, dv, float(m["scale"]),
                                   window=m["window"], sink=w[x + "sink"], gate=proj[:, c:c + H])
        return ops.linear(att, w[x + "o"], w[x + "o.b"])

    def _dense(self, h, p):
        w, F_ = self.w, self.w[p + "down"].shape[1]
        if self.dtype == torch.bfloat16:   # gate / up rows interleaved: the activation is the GEMM's epilogue
            mid = ops.linear(h, w[p + "in"], act="geglu")
        else:
            gu = ops.linear(h, w[p + "in"])
            mid = ops.act_mul(gu[:, :F_], gu[:, F_:], "gelu_tanh", self.dtype)
        return ops.linear(mid, w[p + "down"])

    def _shared(self, h, p, limit):
        """Shared expert -> (output, its gate logit per token): one fused gate | up | sg projection."""
        w, F_ = self.w, self.w[p + "down"].shape[1]
        gu = ops.linear(h, w[p + "in"])
        mid = ops.act_mul(gu[:, :F_], gu[:, F_:2 * F_], "clamp_glu", self.dtype, cap=float(limit))
        return ops.linear(mid, w[p + "down"]), gu[:, 2 * F_:2 * F_ + 1]

    def _moe(self, h, ml, q):
        w, r = self.w, ml["router"]
        E, n = r["experts"], h.shape[0] * r["top"]
        shared = sgate = None
        if ml.get("shared"):
            shared, sgate = self._shared(h, q + "shared.", ml["shared"]["limit"])
        ids, wts = ops.moe_router(h, w[q + "router"], E, r["top"], ROUTE_EPS)
        rows, offs, pos = ops.moe_dispatch(ids, E)
        mid = ops.moe_gemm(h, rows, w[q + "gate_up"], offs, n, act="clamp_glu", act_param=float(ml["expert"]["limit"]))
        out = ops.moe_gemm(mid, None, w[q + "e.down"], offs, n)
        return ops.moe_combine(out, pos, wts, shared, residual_gate=sgate)

    # ------------------------------------------------------------------ forward
    def forward(self, fb: ForwardBatch, kv, decode_ws=None) -> torch.Tensor:
        """Returns fp32 logits [len(sample_rows), vocab]."""
        c, w, dt = self.cfg, self.w, self.dtype
        if fb.extra is None:  # direct forward without the engine hook
            self.prepare_batch(fb)
        seq = dict(fb.extra)
        if "ctx" not in seq:  # captured decode graph: one row per sequence, the engine's static ctx / page tables
            seq["ctx"], seq["bt"] = fb.decode_ctx, fb.decode_block_tables
        eps = c.rms_eps
        res = ops.embed_scale_f32(fb.token_ids, w["embed"], 1.0)
        a = s1 = b = s2 = None      # the previous layer's branch outputs and their scales, not yet in the stream
        for i, t in self.runs:
            p, ml = f"l{i}.", c.layers[i]["mlp"]
            h1, h2 = ops.parallel_add_norm_f32(res, a, s1, b, s2, w[p + "norm1"], w.get(p + "norm2"), eps, dt)
            a, s1 = self._attention(h1, i, (i, t), fb, kv, seq), w[p + "ls1"]
            b = s2 = None
            if ml is not None:
                b = self._moe(h2, ml, p + "mlp.") if ml["kind"] == "moe" else self._dense(h2, p + "mlp.")
                s2 = w[p + "ls2"]
            if self.capture_residuals is not None:
                ops.parallel_add_norm_f32(res, a, s1, b, s2)
                a = s1 = b = s2 = None
                self.capture_residuals.append(res.clone())
        if fb.sample_rows is not None:
            pick = lambda y: None if y is None else y.index_select(0, fb.sample_rows)  # noqa: E731
            res, a, b = pick(res), pick(a), pick(b)
        xf, _ = ops.parallel_add_norm_f32(res, a, s1, b, s2, w["final.norm"], None, eps, dt)
        return ops.linear(xf, w["head"], out_dtype=torch.float32)[:, : c.vocab_size]
