"""A plain, slow float64 implementation of the Bamanex decoder, written from its equations: one function per mechanism,
whole sequences at a time, no cache, no batching. It shares no code with the serving path and is what the tests compare
the framework against.

Notation: x is the residual stream [T, D]; W[name] are the checkpoint tensors (linear weights [out, in], applied as
W x); positions count from 0.
"""
from __future__ import annotations

import math
from typing import Dict, List, Optional

import torch

F64 = torch.float64
ROUTE_EPS = 1e-20        # added to the sum of the chosen router scores
GATE_SLOPE = 1.702       # slope of the sigmoid in the experts' activation


def sigmoid(z):
    return 1.0 / (1.0 + torch.exp(-z))


def gelu_tanh(z):
    return 0.5 * z * (1 + torch.tanh(math.sqrt(2 / math.pi) * (z + 0.044715 * z ** 3)))


def unit_rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def centred_norm(x, w, eps):
    """RMS norm with a zero-centred weight (applied as 1 + w)."""
    return unit_rms(x, eps) * (1 + w)


def frequencies(rot: dict) -> List[float]:
    """Angle per position of every rotated pair: base^(-2i / dims), long waves slowed down by `factor`, with a linear
    cross-over (in turns per `original` positions) between `low` and `high` turns."""
    dims, sc = int(rot.get("dims") or 0), rot.get("scaling")
    out = []
    for i in range(dims // 2):
        f = float(rot["base"]) ** (-2 * i / dims)
        if sc:
            wave, orig = 2 * math.pi / f, float(sc["original"])
            if wave > orig / float(sc["low"]):
                f = f / float(sc["factor"])
            elif wave >= orig / float(sc["high"]):
                s = (orig / wave - float(sc["low"])) / (float(sc["high"]) - float(sc["low"]))
                f = (1 - s) * f / float(sc["factor"]) + s * f
        out.append(f)
    return out


def rotate_halves(x, freqs, positions):
    """x [T, H, d]: channel i < n turned with channel i + n (n = number of frequencies) by position * freqs[i]."""
    n = len(freqs)
    if not n:
        return x
    ang = positions.to(F64)[:, None] * torch.tensor(freqs, dtype=F64)
    c, s = torch.cos(ang)[:, None], torch.sin(ang)[:, None]
    u, v = x[..., :n], x[..., n:2 * n]
    return torch.cat([u * c - v * s, v * c + u * s, x[..., 2 * n:]], -1)


def sink_softmax_head(q, k, v, scale, window, sink, first=0):
    """One head: q [Tq, dk] at positions first .. first + Tq - 1 over k / v of all positions. Position i sees j with
    0 <= i - j < window (0: no lower edge); exp(sink) enters the denominator only."""
    i = torch.arange(first, first + q.shape[0])[:, None]
    j = torch.arange(k.shape[0])[None]
    seen = (j <= i) & ((i - j < window) if window else torch.ones_like(j, dtype=torch.bool))
    s = (q @ k.T) * scale
    top = torch.where(seen, s, torch.full_like(s, -math.inf)).amax(-1, keepdim=True)
    top = torch.clamp(top, min=float(sink))
    e = torch.where(seen, torch.exp(s - top), torch.zeros_like(s))
    return e @ v / (e.sum(-1, keepdim=True) + torch.exp(torch.as_tensor(float(sink), dtype=F64) - top))


def attention_mixer(h, W: Dict[str, torch.Tensor], p: str, m: dict, eps: float):
    H, G, dk, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    T = h.shape[0]
    q, k, v = (h @ W[p + n].T + W[p + n + ".b"] for n in "qkv")
    f, pos = frequencies(m.get("rot") or {}), torch.arange(T)
    q = unit_rms(rotate_halves(q.view(T, H, dk), f, pos), eps)
    k = unit_rms(rotate_halves(k.view(T, G, dk), f, pos), eps)
    v = v.view(T, G, dv)
    gate = sigmoid(h @ W[p + "g"].T)
    window = int((m.get("mask") or {}).get("size") or 0)
    heads = []
    for a in range(H):
        g = a // (H // G)
        o = sink_softmax_head(q[:, a], k[:, g], v[:, g], float(m["scale"]), window, W[p + "sink"][a])
        heads.append(o * gate[:, a:a + 1])
    return torch.cat(heads, -1) @ W[p + "o"].T + W[p + "o.b"]


def dense_ff(h, W, p: str):
    return (gelu_tanh(h @ W[p + "gate"].T) * (h @ W[p + "up"].T)) @ W[p + "down"].T


def clamped_expert(h, W, p: str, limit: float):
    g = torch.clamp(h @ W[p + "gate"].T, max=limit)
    u = torch.clamp(h @ W[p + "up"].T, -limit, limit)
    return (g * sigmoid(GATE_SLOPE * g) * (u + 1)) @ W[p + "down"].T


def route(z, top: int):
    """Router logits -> chosen expert ids [T, top] and weights: softmax scores over all experts, the largest kept and
    divided by their own sum."""
    e = torch.exp(z - z.amax(-1, keepdim=True))
    s = e / e.sum(-1, keepdim=True)
    best, ids = s.topk(top, -1)
    return ids, best / (best.sum(-1, keepdim=True) + ROUTE_EPS)


def moe(h, W, p: str, ml: dict, margins: Optional[list] = None):
    E, top = ml["router"]["experts"], ml["router"]["top"]
    z = h @ W[p + "router"].T
    ids, wts = route(z, top)
    if margins is not None and top < E:
        s = z.sort(-1, descending=True).values
        margins.append((s[:, top - 1] - s[:, top]).min().item())
    out = torch.zeros_like(h)
    for e in range(E):
        share = torch.where(ids == e, wts, torch.zeros_like(wts)).sum(-1)
        rows = share.nonzero().flatten()
        if rows.numel():
            out[rows] += share[rows, None] * clamped_expert(h[rows], W, p + f"e{e}.", float(ml["expert"]["limit"]))
    if ml.get("shared"):
        out = out + clamped_expert(h, W, p + "shared.", float(ml["shared"]["limit"])) * sigmoid(h @ W[p + "shared.sg"].T)
    return out


def layer_order(cfg: dict) -> List[int]:
    n, lp = len(cfg["layers"]), cfg.get("loop")
    if not lp:
        return list(range(n))
    a, b = lp["start"], lp["stop"]
    return list(range(a)) + list(range(a, b)) * lp["times"] + list(range(b, n))


def forward(cfg: dict, sd: Dict[str, torch.Tensor], tokens: List[int], residuals: Optional[list] = None,
            margins: Optional[list] = None):
    """Logits [T, vocab] of one sequence; `residuals` collects the stream after every layer run, `margins` the smallest
    distance between the last chosen and the first rejected router logit of every expert choice."""
    W = {k: torch.as_tensor(v).to(F64) for k, v in sd.items()}
    eps = float(cfg["norm"]["eps"])
    x = W["embed"][torch.as_tensor(tokens, dtype=torch.long)]
    for i in layer_order(cfg):
        l, p = cfg["layers"][i], f"l{i}."
        y = attention_mixer(centred_norm(x, W[p + "norm1"], eps), W, p + "mix.", l["mixer"], eps) * W[p + "ls1"]
        ml = l.get("mlp")
        if ml is not None:   # reads the same x as the mixer
            h = centred_norm(x, W[p + "norm2"], eps)
            y = y + (moe(h, W, p + "mlp.", ml, margins) if ml["kind"] == "moe" else dense_ff(h, W, p + "mlp.")) * W[p + "ls2"]
        x = x + y
        if residuals is not None:
            residuals.append(x.clone())
    return (centred_norm(x, W["final.norm"], eps) @ W["head"].T) * float(cfg.get("logit_scale", 1.0))


# ------------------------------------------------------------------------------------------------ made-up checkpoints
def att(heads=6, kv_heads=2, dim=8, vdim=12, window=11, rot=6, base=50.0, scaling=(3.0, 1.0, 4.0, 40), scale=0.6):
    """scaling: (factor, low, high, original) or None."""
    m = dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, scale=scale, rot=dict(base=base, dims=rot),
             mask=dict(size=window))
    if scaling:
        m["rot"]["scaling"] = dict(zip(("factor", "low", "high", "original"), scaling))
    return dict(type="attention", mixer=m)


def no_ff(layer):
    return dict(layer, mlp=None)


def dense(layer, ff=40):
    return dict(layer, mlp=dict(kind="dense", ff=ff))


def experts(layer, ff=16, n=6, top=2, limit=1.2, shared=24, shared_limit=2.1):
    ml = dict(kind="moe", expert=dict(ff=ff, limit=limit), router=dict(experts=n, top=top))
    if shared:
        ml["shared"] = dict(ff=shared, limit=shared_limit)
    return dict(layer, mlp=ml)


def make_config(layers, width=32, vocab=96, eps=1e-5, logit_scale=0.7, loop=None):
    cfg = dict(architecture="Bamanex", layers=list(layers), norm=dict(eps=eps), vocab=vocab, width=width,
               logit_scale=logit_scale)
    if loop:
        cfg["loop"] = dict(zip(("start", "stop", "times"), loop))
    return cfg


def random_checkpoint(cfg: dict, seed: int) -> Dict[str, torch.Tensor]:
    """bf16-representable random weights with sizeable biases, sinks, gates, norm weights and layer scales."""
    g = torch.Generator().manual_seed(seed)
    D, V = cfg["width"], cfg["vocab"]
    rn = lambda *s: torch.randn(*s, generator=g)  # noqa: E731
    lin = lambda o, i, k=1.0: rn(o, i) * (k * i ** -0.5)  # noqa: E731
    sd = {"embed": rn(V, D), "head": lin(V, D), "final.norm": rn(D) * 0.3}
    for i, l in enumerate(cfg["layers"]):
        p, x, m, ml = f"l{i}.", f"l{i}.mix.", l["mixer"], l.get("mlp")
        H, G, dk, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        for n, rows in (("q", H * dk), ("k", G * dk), ("v", G * dv)):
            sd[x + n], sd[x + n + ".b"] = lin(rows, D), rn(rows) * 0.4
        sd[x + "sink"], sd[x + "g"] = rn(H) * 1.5, lin(H, D, 2.0)
        sd[x + "o"], sd[x + "o.b"] = lin(D, H * dv), rn(D) * 0.3
        sd[p + "norm1"], sd[p + "ls1"] = rn(D) * 0.3, rn(D) * 0.3 + 0.5
        if ml is None:
            continue
        sd[p + "norm2"], sd[p + "ls2"] = rn(D) * 0.3, rn(D) * 0.3 + 0.5
        parts = [("", ml["ff"])] if ml["kind"] == "dense" else [(f"e{e}.", ml["expert"]["ff"])
                                                                for e in range(ml["router"]["experts"])]
        if ml["kind"] == "moe":
            sd[p + "mlp.router"] = lin(ml["router"]["experts"], D, 1.5)
            if ml.get("shared"):
                parts.append(("shared.", ml["shared"]["ff"]))
                sd[p + "mlp.shared.sg"] = lin(1, D, 2.0)
        for n, F_ in parts:
            q = p + "mlp." + n
            sd[q + "gate"], sd[q + "up"], sd[q + "down"] = lin(F_, D, 1.5), lin(F_, D, 1.5), lin(D, F_)
    return {k: v.to(torch.bfloat16).float() for k, v in sd.items()}
