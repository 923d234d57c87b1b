"""Luketar: a hybrid decoder whose layer list mixes latent attention and matrix-memory LSTM layers, with several residual
streams joined by hyper-connections, layer norms, and dense or mixture-of-experts feed-forwards.

Architecture (every size and constant comes from ``config.json``; the layer list may hold the mixers in any order):
  * token embedding times a scale; the output head is the embedding table itself (without the scale);
  * ``streams`` residual streams X_1 .. X_s, all equal to the embedding output at first. A sublayer (mixer, feed-forward) reads
    ``u = sum_s in[s] X_s`` through a layer norm (weight, no bias) and its output y goes back as
    ``X_t <- sum_s mix[s, t] X_s + out[t] y``; after the last layer the streams are summed;
  * a layer may have no feed-forward, and may use the weights of another one (``weights_of``) with a cache / state of its
    own;
  * mixer ``latent_attention``: queries from a normed low-rank latent of their own, keys and values linear maps of one normed
    latent per token (all of the cache), no positions, causal softmax with a learned value-less sink score per head, the
    heads' outputs times ``sigmoid(W_g h)``;
  * mixer ``mlstm``: matrix memory ``S <- e^f S + e^i k v^T`` with capped exponential gates per head, kept in range by a
    running maximum, a normaliser state, a per-head RMS norm and a sigmoid gate;
  * feed-forward ``dense``: ``W_down (g sigmoid(1.702 g) (u + 1))`` with ``g = min(W_gate h, limit)``, ``u = clamp(W_up h, +-limit)``;
    ``moe``: experts of that form, the ``top`` largest router logits (with a bias) chosen, weights = softmax over the chosen
    logits, plus an always-on shared expert.

MI355X mapping: residual streams, norms, attention scores and weights, router, gates and recurrent states are fp32;
projections run in the model dtype on the MFMA GEMMs (bf16 with fp32 accumulation, or true fp32). One kernel between two
sublayers mixes the streams, adds the output, reads the next input and norms it. Latent attention folds the queries
through the key expansion and attends over the cached latents with one kv head (the paged window kernels). The matrix
memory runs chunk by chunk on the fp32 matrix cores with its state in accumulator registers, and as one fused kernel per
(sequence, head) in decode steps. A step's rows - prompt portions and single decoded tokens alike - are addressed by
device-side (cu, slot, ctx) vectors, so pure-decode steps replay a captured HIP graph.
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
from .hybrid_base import HybridDecoderBase, stack_gated_experts

MIXERS = ("latent_attention", "mlstm")
DEN_EPS = 1e-6         # added to the matrix memory's denominator


@dataclass
class LuketarConfig:
    vocab_size: int
    hidden_size: int
    layers: Tuple[dict, ...]     # {"type", "mixer": {...}, "mlp": {"kind": "dense" | "moe", ...} | None, "weights_of"?: j}
    streams: int = 1
    embed_scale: float = 1.0
    norm_eps: float = 1e-6
    name: str = "luketar"
    max_position: int = 1 << 20              # no positions enter: nothing to outgrow
    bos_token_id: Optional[int] = None
    eos_token_ids: Tuple[int, ...] = ()

    def __post_init__(self):
        if self.streams < 1:
            raise ValueError("streams must be >= 1")
        layers = []
        for i, l in enumerate(self.layers):
            if l["type"] not in MIXERS:
                raise ValueError(f"layer {i}: unknown mixer type {l['type']!r}")
            m = dict(l["mixer"])
            m.setdefault("vdim", m["dim"])
            if l["type"] == "latent_attention":
                m.setdefault("scale", m["dim"] ** -0.5)
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
        for i, l in enumerate(layers):
            if l.get("weights_of") is None:
                continue
            j = self.weight_layer(i)
            if layers[j]["type"] != l["type"] or layers[j]["mixer"] != l["mixer"] or layers[j]["mlp"] != l["mlp"]:
                raise ValueError(f"layer {i}: differs from layer {j}, whose weights it uses")

    @property
    def num_layers(self) -> int:
        return len(self.layers)

    @property
    def head_dim(self) -> int:  # engine sizing hooks: the widest cached key row
        return max([l["mixer"]["kv_rank"] for l in self.layers if l["type"] == "latent_attention"] or [16])

    def weight_layer(self, i: int) -> int:
        """The layer whose tensors layer i uses."""
        j, hops = i, 0
        while self.layers[j].get("weights_of") is not None:
            j, hops = int(self.layers[j]["weights_of"]), hops + 1
            if not 0 <= j < len(self.layers) or hops > len(self.layers):
                raise ValueError(f"layer {i}: weights_of does not lead to a layer with weights of its own")
        return j

    @staticmethod
    def from_json(path_or_dict) -> "LuketarConfig":
        if isinstance(path_or_dict, dict):
            c, name = path_or_dict, "luketar"
        else:
            with open(os.path.join(path_or_dict, "config.json")) as f:
                c = json.load(f)
            name = os.path.basename(os.path.normpath(path_or_dict)) or "luketar"
        eos = c.get("eos_token_id", ())
        return LuketarConfig(
            vocab_size=int(c["vocab"]), hidden_size=int(c["width"]), layers=tuple(c["layers"]),
            streams=int(c.get("streams", 1)), embed_scale=float((c.get("embedding") or {}).get("scale", 1.0)),
            norm_eps=float((c.get("norm") or {}).get("eps", 1e-6)),
            name=c.get("name", name), max_position=int(c.get("max_position", 1 << 20)),
            bos_token_id=c.get("bos_token_id"), eos_token_ids=tuple(eos) if isinstance(eos, (list, tuple)) else (eos,))

    @staticmethod
    def tiny(**kw) -> "LuketarConfig":
        att = dict(heads=2, dim=16, vdim=24, q_rank=48, kv_rank=40, scale=0.3)
        mem = dict(heads=2, dim=16, vdim=24, gate_cap=10.0)
        dense = dict(kind="dense", ff=96, limit=3.0)
        moe = dict(kind="moe", expert=dict(ff=32, limit=2.0), shared=dict(ff=48, limit=3.0), router=dict(experts=6, top=2))
        base = dict(vocab_size=512, hidden_size=64, name="tiny-luketar", norm_eps=1e-5, streams=3, embed_scale=2.0,
                    layers=(dict(type="mlstm", mixer=mem, mlp=dense), dict(type="latent_attention", mixer=att, mlp=moe),
                            dict(type="mlstm", mixer=mem, mlp=None),
                            dict(type="latent_attention", mixer=att, mlp=moe, weights_of=1)))
        base.update(kw)
        return LuketarConfig(**base)

    @staticmethod
    def sized(width: int, n_layers: int, ff: int, heads: int, head_dim: int, vocab: int = 32768, experts: int = 8,
              top: int = 2, pattern: Tuple[str, ...] = MIXERS, **kw) -> "LuketarConfig":
        """A regular stack for benchmarks: `pattern` repeated over n_layers; key / value latents of two heads' size, query
        latents of half the width; every layer carries `experts` experts of ff / top (the active routed feed-forward
        equals a dense ff) plus a shared expert of ff / 4."""
        mix = dict(latent_attention=dict(heads=heads, dim=head_dim, vdim=head_dim, q_rank=width // 2, kv_rank=2 * head_dim,
                                         scale=head_dim ** -0.5),
                   mlstm=dict(heads=heads, dim=head_dim, vdim=head_dim, gate_cap=15.0))
        moe = dict(kind="moe", expert=dict(ff=ff // top, limit=7.0), shared=dict(ff=ff // 4, limit=7.0),
                   router=dict(experts=experts, top=top))
        layers = tuple(dict(type=pattern[i % len(pattern)], mixer=mix[pattern[i % len(pattern)]], mlp=moe)
                       for i in range(n_layers))
        base = dict(vocab_size=vocab, hidden_size=width, layers=layers, streams=4, name=f"luketar-{width}x{n_layers}")
        base.update(kw)
        return LuketarConfig(**base)


def random_state(cfg: LuketarConfig, seed: int = 0) -> Dict[str, torch.Tensor]:
    """A random checkpoint (tensor names and shapes of the safetensors layout, fp32 values) with magnitudes that keep
    activations, gates and states in a trained model's range."""
    g = torch.Generator().manual_seed(seed)
    D, ns = cfg.hidden_size, cfg.streams
    rn = lambda *s, std=1.0: torch.randn(*s, generator=g) * std  # noqa: E731
    un = lambda *s, lo=0.0, hi=1.0: torch.rand(*s, generator=g) * (hi - lo) + lo  # noqa: E731
    lin = lambda o, i: rn(o, i, std=i ** -0.5)  # noqa: E731
    sd: Dict[str, torch.Tensor] = {"embed": rn(cfg.vocab_size, D), "final.norm": 1 + rn(D, std=0.1)}

    def gated(p, F_):
        sd[p + "gate"], sd[p + "up"], sd[p + "down"] = lin(F_, D) * 1.5, lin(F_, D), lin(D, F_)

    for i, l in enumerate(cfg.layers):
        if l.get("weights_of") is not None:
            continue
        p, m, x = f"l{i}.", l["mixer"], f"l{i}.mix."
        for q in (1, 2) if l.get("mlp") is not None else (1,):
            sd[p + f"norm{q}"] = 1 + rn(D, std=0.1)
            sd[p + f"hc{q}.in"], sd[p + f"hc{q}.out"] = un(ns, lo=0.2, hi=1.0) / ns ** 0.5, un(ns, lo=0.3, hi=1.0)
            sd[p + f"hc{q}.mix"] = torch.eye(ns) * 0.9 + rn(ns, ns, std=0.1)
        H, dk, dv = m["heads"], m["dim"], m["vdim"]
        if l["type"] == "latent_attention":
            rq, rk = m["q_rank"], m["kv_rank"]
            sd[x + "dq"], sd[x + "dq.norm"], sd[x + "uq"] = lin(rq, D), 1 + rn(rq, std=0.1), lin(H * dk, rq) * 2.0
            sd[x + "dkv"], sd[x + "dkv.norm"] = lin(rk, D), 1 + rn(rk, std=0.1)
            sd[x + "uk"], sd[x + "uv"], sd[x + "sink"] = lin(H * dk, rk), lin(H * dv, rk), rn(H)
        else:
            sd[x + "q"], sd[x + "k"], sd[x + "v"] = lin(H * dk, D), lin(H * dk, D), lin(H * dv, D)
            sd[x + "i"], sd[x + "i.b"] = lin(H, D), rn(H, std=0.3)
            sd[x + "f"], sd[x + "f.b"] = lin(H, D), un(H, lo=1.0, hi=6.0)
            sd[x + "norm"] = 1 + rn(H * dv, std=0.1)
        sd[x + "g"], sd[x + "o"] = lin(H * dv, D), lin(D, H * dv)
        ml = l.get("mlp")
        if ml is None:
            continue
        if ml["kind"] == "dense":
            gated(p + "mlp.", ml["ff"])
            continue
        r = ml["router"]
        for e in range(r["experts"]):
            gated(p + f"mlp.e{e}.", ml["expert"]["ff"])
        sd[p + "mlp.router"], sd[p + "mlp.router.b"] = lin(r["experts"], D), rn(r["experts"], std=0.2)
        if ml.get("shared"):
            gated(p + "mlp.shared.", ml["shared"]["ff"])
    return sd


class LuketarModel(HybridDecoderBase):
    """Weights (plain tensors) + forward for the serving engine (the hooks of LlamaModel / PinavikModel)."""

    def __init__(self, cfg: LuketarConfig, device=None, dtype=torch.bfloat16, dist_ctx: DistContext | None = None,
                 state_slots: Optional[int] = None):
        self.cfg = cfg
        self.ctx = dist_ctx or get_context()
        assert self.ctx.tp_size == 1, "Luketar runs TP=1"
        self.device = torch.device(device) if device is not None else self.ctx.device
        self.dtype = dtype
        att = [i for i, l in enumerate(cfg.layers) if l["type"] == "latent_attention"]
        self.kv_index = {i: j for j, i in enumerate(att)}
        self.num_kv_layers = len(att)
        self.hq = max([cfg.layers[i]["mixer"]["heads"] for i in att] or [1])
        self.hkv = 1
        self.vocab_local, self.vstart = cfg.vocab_size, 0
        self.lora_names: list = []
        self.w: Dict[str, torch.Tensor] = {}
        self.pool = StatePool(state_slots or int(os.environ.get("GAI_LINEAR_STATE_SLOTS", "64")), self.device)
        self.state: Dict[int, Dict[str, torch.Tensor]] = {}
        self.capture_residuals: Optional[list] = None  # numerics debugging: the sum of the streams after every layer

    # ------------------------------------------------------------------ engine sizing hooks
    def kv_layout(self) -> List[Tuple[int, int, int]]:
        """(kv heads, key size, value size) of every paged cache layer: one per latent-attention layer, ONE kv head whose
        key row and value row are the latent."""
        out = []
        for i in sorted(self.kv_index, key=self.kv_index.get):
            r = self.cfg.layers[i]["mixer"]["kv_rank"]
            out.append((1, r, r))
        return out

    # ------------------------------------------------------------------ weights
    def load_state(self, sd: Dict[str, torch.Tensor]):
        """Checkpoint tensors (the safetensors names) -> device weights: projections in the model dtype, per-channel
        tables fp32, same-input projections fused, expert matrices stacked with gate / up rows interleaved per 16 (rows
        padded with zeros to the grouped GEMM's grid: a zero gate row contributes nothing)."""
        c, dev, dt = self.cfg, self.device, self.dtype
        f32 = lambda t: t.to(torch.float32).to(dev).contiguous()  # noqa: E731
        mat = lambda t: t.to(torch.float32).to(dev, dt).contiguous()  # noqa: E731
        pad16 = lambda t: torch.cat([t.float(), torch.zeros((-t.shape[0]) % 16, t.shape[1])])  # noqa: E731
        D = c.hidden_size
        w = self.w = {}
        w["embed"] = mat(pad16(sd["embed"]))     # padded rows: columns of the logits that forward() cuts off
        w["final.norm"], w["final.in"] = f32(sd["final.norm"]), torch.ones(c.streams, device=dev)
        for i, l in enumerate(c.layers):
            if l.get("weights_of") is not None:
                continue
            p, x, m = f"l{i}.", f"l{i}.mix.", l["mixer"]
            ml = l.get("mlp")
            for q in (1, 2) if ml is not None else (1,):
                w[p + f"norm{q}"] = f32(sd[p + f"norm{q}"])
                for n in ("in", "out", "mix"):
                    w[p + f"hc{q}.{n}"] = f32(sd[p + f"hc{q}.{n}"])
            H = m["heads"]
            if l["type"] == "latent_attention":
                w[x + "in"] = mat(pad16(torch.cat([sd[x + k].float() for k in ("dq", "dkv", "g")])))
                w[x + "dq.norm"], w[x + "dkv.norm"], w[x + "sink"] = f32(sd[x + "dq.norm"]), f32(sd[x + "dkv.norm"]), f32(sd[x + "sink"])
                w[x + "uq"] = mat(sd[x + "uq"])
                w[x + "uk"] = mat(sd[x + "uk"].float().reshape(H, m["dim"], m["kv_rank"]).transpose(1, 2))  # [H, kv_rank, dim]
                w[x + "uv"] = mat(sd[x + "uv"].float().reshape(H, m["vdim"], m["kv_rank"]))
            else:
                w[x + "in"] = mat(pad16(torch.cat([sd[x + k].float() for k in ("q", "k", "v", "g")])))
                w[x + "if"] = mat(pad16(torch.cat([sd[x + k].float() for k in ("i", "f")])))
                w[x + "i.b"], w[x + "f.b"], w[x + "norm"] = f32(sd[x + "i.b"]), f32(sd[x + "f.b"]), f32(sd[x + "norm"])
            w[x + "o"] = mat(sd[x + "o"])
            if ml is None:
                continue
            q = p + "mlp."
            def plain_ff(src, dst):
                # wide feed-forwards padded with zeros to the split-K decode GEMM's grid (a zero gate row contributes nothing)
                F_ = sd[src + "gate"].shape[0]
                z = torch.zeros((-F_) % 512 if dt == torch.bfloat16 and F_ >= 1024 else 0, D)
                w[dst + "in"] = mat(pad16(torch.cat([sd[src + "gate"].float(), z, sd[src + "up"].float(), z])))
                w[dst + "down"] = mat(torch.cat([sd[src + "down"].float(), z.t()], 1))

            if ml["kind"] == "dense":
                plain_ff(q, q)
                continue
            E = ml["router"]["experts"]
            # router rows padded to the GEMM's 16-column grid: the logits come out of the MFMA kernel in fp32
            w[q + "router"], w[q + "router.b"] = mat(pad16(sd[q + "router"])), f32(sd[q + "router.b"])
            gate_up, down = stack_gated_experts(sd, q, E, 64 if dt == torch.bfloat16 else 16)
            w[q + "gate_up"], w[q + "e.down"] = mat(gate_up), mat(down)
            if ml.get("shared"):
                plain_ff(q + "shared.", q + "shared.")
        self._alloc_state()
        return self

    def random_init(self, seed: int = 0):
        return self.load_state(random_state(self.cfg, seed))

    # ------------------------------------------------------------------ recurrent state slots
    def _alloc_state(self):
        self.pool.clear()
        self.state = {}
        for i, l in enumerate(self.cfg.layers):
            if l["type"] == "mlstm":
                m, tag = l["mixer"], f"l{i}."
                self.state[i] = dict(S=self.pool.add(tag + "S", (m["heads"], m["dim"], m["vdim"])),
                                     n=self.pool.add(tag + "n", (m["heads"], m["dim"])),
                                     m=self.pool.add(tag + "m", (m["heads"],)))

    # ------------------------------------------------------------------ mixers
    def _latent_attention(self, h, i, x, fb, kv, seq):
        m, w = self.cfg.layers[i]["mixer"], self.w
        H, rq, rk = m["heads"], m["q_rank"], m["kv_rank"]
        nv = H * m["vdim"]
        proj = ops.linear(h, w[x + "in"])
        kc, vc = kv.layer(self.kv_index[i])
        cq = ops.latent_norm_write(proj[:, :rq], w[x + "dq.norm"], proj[:, rq:rq + rk], w[x + "dkv.norm"], fb.slots, kc, vc,
                                   self.cfg.norm_eps)
        # the queries folded through the key expansion: scores against the cached latent need no keys
        qf = ops.head_linear(ops.linear(cq, w[x + "uq"]), w[x + "uk"])
        lat = ops.window_attention(qf, kc, vc, seq["bt"], seq["cu"], seq["ctx"], H, 1, rk, rk, float(m["scale"]),
                                   sink=w[x + "sink"])
        # the weighted latents expanded to the heads' values, gated
        return ops.linear(ops.head_linear(lat, w[x + "uv"], proj[:, rq + rk:rq + rk + nv]), w[x + "o"])

    def _mlstm(self, h, i, x, seq):
        m, w, st = self.cfg.layers[i]["mixer"], self.w, self.state[i]
        H, dk, dv = m["heads"], m["dim"], m["vdim"]
        a, b = 2 * H * dk, 2 * H * dk + H * dv
        proj = ops.linear(h, w[x + "in"])
        gl = ops.linear(h, w[x + "if"], out_dtype=torch.float32)
        y = ops.mlstm(proj[:, :H * dk], proj[:, H * dk:a], proj[:, a:b], gl[:, :H], gl[:, H:2 * H], w[x + "i.b"],
                      w[x + "f.b"], float(m["gate_cap"]), proj[:, b:b + H * dv], w[x + "norm"], st["S"], st["n"], st["m"],
                      seq["cu"], seq["slots"], dk ** -0.5, self.cfg.norm_eps, DEN_EPS, self.dtype)
        return ops.linear(y, w[x + "o"])

    # ------------------------------------------------------------------ feed-forwards
    def _gated(self, h, w_in, w_down, limit):
        """W_down of the clamped gated activation of one fused gate | up projection."""
        F_ = w_down.shape[1]
        gu = ops.linear(h, w_in)
        return ops.linear(ops.act_mul(gu[:, :F_], gu[:, F_:2 * F_], "clamp_glu", self.dtype, cap=float(limit)), w_down)

    def _moe(self, h, ml, q):
        w, r = self.w, ml["router"]
        E, top = r["experts"], r["top"]
        logits = ops.linear(h, w[q + "router"], out_dtype=torch.float32)[:, :E]
        ids, wts = ops.moe_route(logits, top, score="chosen", bias=w[q + "router.b"])
        shared = self._gated(h, w[q + "shared.in"], w[q + "shared.down"], ml["shared"]["limit"]) if ml.get("shared") else None
        rows, offs, pos = ops.moe_dispatch(ids, E)
        n = h.shape[0] * top
        mid = ops.moe_gemm(h, rows, w[q + "gate_up"], offs, n, act="clamp_glu", act_param=float(ml["expert"]["limit"]))
        return ops.moe_combine(ops.moe_gemm(mid, None, w[q + "e.down"], offs, n), pos, wts, shared)

    # ------------------------------------------------------------------ forward
    def forward(self, fb: ForwardBatch, kv, decode_ws=None) -> torch.Tensor:
        """Returns fp32 logits [len(sample_rows), vocab]."""
        c, w, dt = self.cfg, self.w, self.dtype
        if fb.extra is None:  # direct forward without the engine hook
            self.prepare_batch(fb)
        seq = dict(fb.extra)
        if "ctx" not in seq:  # captured decode graph: one row per sequence, the engine's static ctx / page tables
            seq["ctx"], seq["bt"] = fb.decode_ctx, fb.decode_block_tables
        eps = c.norm_eps
        x0 = ops.embed_scale_f32(fb.token_ids, w["embed"], c.embed_scale)
        X = torch.empty(x0.shape[0], c.streams, x0.shape[1], dtype=torch.float32, device=x0.device)
        first, y, closing = x0, None, None    # y: output of the sublayer whose weights `closing` names

        def between(in_w, norm_w):
            """Close the previous sublayer, open the next one (in_w None: only close)."""
            nonlocal first, y
            mix, out_w = (w[closing + "mix"], w[closing + "out"]) if y is not None else (None, None)
            h = ops.hyper_connect(X, first, y, mix, out_w, in_w, norm_w, eps, dt)
            first = y = None
            return h

        for i, l in enumerate(c.layers):
            p = f"l{c.weight_layer(i)}."
            h = between(w[p + "hc1.in"], w[p + "norm1"])
            y = self._latent_attention(h, i, p + "mix.", fb, kv, seq) if l["type"] == "latent_attention" \
                else self._mlstm(h, i, p + "mix.", seq)
            closing = p + "hc1."
            ml = l.get("mlp")
            if ml is not None:
                h = between(w[p + "hc2.in"], w[p + "norm2"])
                y = self._moe(h, ml, p + "mlp.") if ml["kind"] == "moe" else \
                    self._gated(h, w[p + "mlp.in"], w[p + "mlp.down"], ml["limit"])
                closing = p + "hc2."
            if self.capture_residuals is not None:
                between(None, None)
                self.capture_residuals.append(X.sum(1))
        if fb.sample_rows is not None:
            rows = fb.sample_rows
            X, first, y = X.index_select(0, rows), first if first is None else first.index_select(0, rows), \
                y if y is None else y.index_select(0, rows)
        xf = between(w["final.in"], w["final.norm"])
        return ops.linear(xf, w["embed"], out_dtype=torch.float32)[:, : c.vocab_size]
