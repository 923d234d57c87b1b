"""A plain, slow float64 implementation of the Luketar decoder, written from its equations: one function per mechanism,
whole sequences at a time, no cache, no batching. It shares no code with the serving path and is what the tests compare
the framework against.

Notation: X is the list of residual streams, each [T, D]; W[name] are the checkpoint tensors (linear weights [out, in],
applied as W x).
"""
from __future__ import annotations

import math
from typing import Dict, List, Optional

import torch

F64 = torch.float64
DEN_EPS = 1e-6           # added to the matrix memory's denominator
GATE_SLOPE = 1.702       # slope of the sigmoid in the feed-forward activation


def t64(t) -> torch.Tensor:
    return torch.as_tensor(t).to(F64)


def layer_norm(x, w, eps):
    d = x - x.mean(-1, keepdim=True)
    return d / torch.sqrt((d * d).mean(-1, keepdim=True) + eps) * w


def unit_rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def sigmoid(z):
    return 1 / (1 + torch.exp(-z))


def read_streams(X: List[torch.Tensor], w_in):
    return sum(w_in[s] * X[s] for s in range(len(X)))


def write_streams(X: List[torch.Tensor], mix, w_out, y):
    """All streams at once, from the old ones; mix is indexed [from, to]."""
    n = len(X)
    return [sum(mix[s, t] * X[s] for s in range(n)) + w_out[t] * y for t in range(n)]


def mlstm_cell(q, k, v, i, f, S, n, m):
    """Matrix memory of one head over a sequence: q (scaled) / k [T, dk], v [T, dv], log gates i / f [T], starting from
    (S, n, m). Returns the outputs before the head norm and the final state."""
    out = []
    for t in range(q.shape[0]):
        m_new = torch.maximum(f[t] + m, i[t])
        keep, put = torch.exp(f[t] + m - m_new), torch.exp(i[t] - m_new)
        S = keep * S + put * torch.outer(k[t], v[t])
        n = keep * n + put * k[t]
        m = m_new
        out.append((S.T @ q[t]) / (torch.maximum((n @ q[t]).abs(), torch.exp(-m)) + DEN_EPS))
    return torch.stack(out), S, n, m


def log_gates(zi, zf, cap):
    """Capped log input gate and log forget gate from their biased logits."""
    soft = lambda z: cap * torch.tanh(z / cap)  # noqa: E731
    return soft(zi), -torch.log1p(torch.exp(-soft(zf)))


def mlstm_mixer(h, W: Dict[str, torch.Tensor], p: str, m: dict, eps: float):
    H, dk, dv, T = m["heads"], m["dim"], m["vdim"], h.shape[0]
    q = (h @ W[p + "q"].T).view(T, H, dk) * dk ** -0.5
    k = (h @ W[p + "k"].T).view(T, H, dk)
    v = (h @ W[p + "v"].T).view(T, H, dv)
    i, f = log_gates(h @ W[p + "i"].T + W[p + "i.b"], h @ W[p + "f"].T + W[p + "f.b"], float(m["gate_cap"]))
    o = torch.stack([mlstm_cell(q[:, j], k[:, j], v[:, j], i[:, j], f[:, j], torch.zeros(dk, dv, dtype=F64),
                                torch.zeros(dk, dtype=F64), torch.zeros((), dtype=F64))[0] for j in range(H)], 1)
    y = unit_rms(o, eps).reshape(T, H * dv) * W[p + "norm"] * sigmoid(h @ W[p + "g"].T)
    return y @ W[p + "o"].T


def sink_softmax(s, sink):
    """Softmax over the last axis whose denominator also holds exp(sink)."""
    top = torch.maximum(s.max(-1, keepdim=True).values, sink)
    e = torch.exp(s - top)
    return e / (e.sum(-1, keepdim=True) + torch.exp(sink - top))


def latent_attention_mixer(h, W, p, m, eps):
    H, dk, dv, T = m["heads"], m["dim"], m["vdim"], h.shape[0]
    cq = unit_rms(h @ W[p + "dq"].T, eps) * W[p + "dq.norm"]
    q = (cq @ W[p + "uq"].T).view(T, H, dk)
    c = unit_rms(h @ W[p + "dkv"].T, eps) * W[p + "dkv.norm"]
    k = (c @ W[p + "uk"].T).view(T, H, dk)
    v = (c @ W[p + "uv"].T).view(T, H, dv)
    hidden = torch.ones(T, T).triu(1).bool()
    out = []
    for j in range(H):
        s = (q[:, j] @ k[:, j].T * float(m["scale"])).masked_fill(hidden, -math.inf)
        out.append(sink_softmax(s, W[p + "sink"][j]) @ v[:, j])
    return (torch.cat(out, 1) * sigmoid(h @ W[p + "g"].T)) @ W[p + "o"].T


def gated_ff(h, W, p, limit):
    g = (h @ W[p + "gate"].T).clamp(max=limit)
    u = (h @ W[p + "up"].T).clamp(-limit, limit)
    return (g * sigmoid(GATE_SLOPE * g) * (u + 1)) @ W[p + "down"].T


def router_logits(h, W, p):
    return h @ W[p + "router"].T + W[p + "router.b"]


def moe_ff(h, W, p, ml):
    r = ml["router"]
    z, ids = router_logits(h, W, p).topk(r["top"], -1)
    w = torch.softmax(z, -1)
    out = torch.zeros_like(h)
    for e in range(r["experts"]):
        we = (w * (ids == e)).sum(-1, keepdim=True)
        out = out + we * gated_ff(h, W, p + f"e{e}.", float(ml["expert"]["limit"]))
    if ml.get("shared"):
        out = out + gated_ff(h, W, p + "shared.", float(ml["shared"]["limit"]))
    return out


def forward(cfg: dict, sd: Dict[str, torch.Tensor], toks, residuals: Optional[list] = None, margins: Optional[list] = None):
    """Logits [T, vocab]; residuals: the sum of the streams after every layer; margins: per routed layer the smallest
    gap between the last chosen and the first rejected router logit."""
    W = {k: t64(v) for k, v in sd.items()}
    eps = float(cfg["norm"]["eps"])
    x = W["embed"][torch.as_tensor(toks)] * float(cfg["embedding"]["scale"])
    X = [x for _ in range(cfg["streams"])]
    for i, l in enumerate(cfg["layers"]):
        j = i
        while cfg["layers"][j].get("weights_of") is not None:
            j = cfg["layers"][j]["weights_of"]
        p = f"l{j}."
        h = layer_norm(read_streams(X, W[p + "hc1.in"]), W[p + "norm1"], eps)
        mixer = latent_attention_mixer if l["type"] == "latent_attention" else mlstm_mixer
        X = write_streams(X, W[p + "hc1.mix"], W[p + "hc1.out"], mixer(h, W, p + "mix.", l["mixer"], eps))
        ml = l["mlp"]
        if ml is not None:
            h = layer_norm(read_streams(X, W[p + "hc2.in"]), W[p + "norm2"], eps)
            if ml["kind"] == "dense":
                y = gated_ff(h, W, p + "mlp.", float(ml["limit"]))
            else:
                y = moe_ff(h, W, p + "mlp.", ml)
                r = ml["router"]
                if margins is not None and r["top"] < r["experts"]:
                    z = router_logits(h, W, p + "mlp.").sort(-1, descending=True).values
                    margins.append(float((z[:, r["top"] - 1] - z[:, r["top"]]).min()))
            X = write_streams(X, W[p + "hc2.mix"], W[p + "hc2.out"], y)
        if residuals is not None:
            residuals.append(sum(X))
    return layer_norm(sum(X), W["final.norm"], eps) @ W["embed"].T


# ------------------------------------------------------------------------------------------------ made-up models
def att(heads=4, dim=10, vdim=14, q_rank=18, kv_rank=26, scale=0.4):
    return "latent_attention", dict(heads=heads, dim=dim, vdim=vdim, q_rank=q_rank, kv_rank=kv_rank, scale=scale)


def mem(heads=3, dim=12, vdim=20, gate_cap=8.0):
    return "mlstm", dict(heads=heads, dim=dim, vdim=vdim, gate_cap=gate_cap)


def no_ff(mixer):
    return dict(type=mixer[0], mixer=mixer[1], mlp=None)


def dense(mixer, ff=36, limit=1.5):
    return dict(type=mixer[0], mixer=mixer[1], mlp=dict(kind="dense", ff=ff, limit=limit))


def moe(mixer, ff=24, experts=6, top=2, limit=1.2, shared=20, shared_limit=0.9):
    ml = dict(kind="moe", expert=dict(ff=ff, limit=limit), router=dict(experts=experts, top=top))
    if shared:
        ml["shared"] = dict(ff=shared, limit=shared_limit)
    return dict(type=mixer[0], mixer=mixer[1], mlp=ml)


def again(layer, j):
    return dict(layer, weights_of=j)


def make_config(layers, width=40, vocab=120, streams=3, scale=1.7, eps=1e-5):
    return dict(architecture="Luketar", vocab=vocab, width=width, layers=list(layers), streams=streams,
                embedding=dict(scale=scale), norm=dict(eps=eps))


def random_checkpoint(cfg, seed, slow_forget=False):
    """Random weights with sinks, biases, stream weights and gates of sizeable spread, rounded to bf16 values (so that a
    bf16 and an fp32 model hold the same numbers). slow_forget: forget gates near one (a long memory)."""
    g = torch.Generator().manual_seed(seed)
    rn = lambda *s, std=1.0: torch.randn(*s, generator=g) * std  # noqa: E731
    un = lambda *s, lo=0.0, hi=1.0: torch.rand(*s, generator=g) * (hi - lo) + lo  # noqa: E731
    lin = lambda o, i, gain=1.0: rn(o, i, std=gain * i ** -0.5)  # noqa: E731
    D, ns = cfg["width"], cfg["streams"]
    sd = {"embed": rn(cfg["vocab"], D), "final.norm": 1 + rn(D, std=0.2)}

    def ff(p, F_):
        sd[p + "gate"], sd[p + "up"], sd[p + "down"] = lin(F_, D, 1.5), lin(F_, D, 1.5), lin(D, F_)

    for i, l in enumerate(cfg["layers"]):
        if l.get("weights_of") is not None:
            continue
        p, x, m, ml = f"l{i}.", f"l{i}.mix.", l["mixer"], l["mlp"]
        for q in (1, 2) if ml is not None else (1,):
            sd[p + f"norm{q}"] = 1 + rn(D, std=0.2)
            sd[p + f"hc{q}.in"], sd[p + f"hc{q}.out"] = rn(ns, std=0.3) + 0.5, rn(ns, std=0.3) + 0.7
            sd[p + f"hc{q}.mix"] = torch.eye(ns) * 0.8 + rn(ns, ns, std=0.2)
        H, dk, dv = m["heads"], m["dim"], m["vdim"]
        if l["type"] == "latent_attention":
            rq, rk = m["q_rank"], m["kv_rank"]
            sd[x + "dq"], sd[x + "dq.norm"], sd[x + "uq"] = lin(rq, D), 1 + rn(rq, std=0.2), lin(H * dk, rq, 2.0)
            sd[x + "dkv"], sd[x + "dkv.norm"] = lin(rk, D), 1 + rn(rk, std=0.2)
            sd[x + "uk"], sd[x + "uv"], sd[x + "sink"] = lin(H * dk, rk, 1.5), lin(H * dv, rk), rn(H, std=1.5) + 1.0
        else:
            sd[x + "q"], sd[x + "k"], sd[x + "v"] = lin(H * dk, D), lin(H * dk, D), lin(H * dv, D)
            sd[x + "i"], sd[x + "i.b"] = lin(H, D, 1.5), rn(H)
            sd[x + "f"], sd[x + "f.b"] = lin(H, D), un(H, lo=0.0, hi=4.0)
            if slow_forget:
                sd[x + "f"], sd[x + "f.b"] = sd[x + "f"] * 0.2, un(H, lo=6.0, hi=8.0)
            sd[x + "norm"] = 1 + rn(H * dv, std=0.2)
        sd[x + "g"], sd[x + "o"] = lin(H * dv, D), lin(D, H * dv)
        if ml is None:
            continue
        if ml["kind"] == "dense":
            ff(p + "mlp.", ml["ff"])
            continue
        E = ml["router"]["experts"]
        for e in range(E):
            ff(p + f"mlp.e{e}.", ml["expert"]["ff"])
        sd[p + "mlp.router"], sd[p + "mlp.router.b"] = lin(E, D, 1.5), rn(E)
        if ml.get("shared"):
            ff(p + "mlp.shared.", ml["shared"]["ff"])
    return {k: v.to(torch.bfloat16).float() for k, v in sd.items()}
