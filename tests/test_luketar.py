"""Luketar decoder: the framework (model registry -> LLMEngine -> native scheduler -> ops) against the slow float64 oracle
in tests/luketar_oracle.py. Small made-up configurations and random weights with sizeable sinks, biases, stream weights
and gates, so that a lost state, a wrong stream, a sink left out, a wrong expert or a wrong page moves the logits far
beyond the tolerance. CPU runs use the reference ops, GPU runs the HIP kernels (fp32: tight tolerance; bf16: rounding
level).
"""
import json
import math
import os
import subprocess
import sys

import pytest
import torch

from generativeaiexamples_amd import ops
from generativeaiexamples_amd.engine import EngineConfig, LLMEngine, SamplingParams
from generativeaiexamples_amd.models.luketar import DEN_EPS, LuketarConfig, LuketarModel
from generativeaiexamples_amd.models.registry import build_llm

from . import luketar_oracle as O

_GPU = pytest.mark.gpu
TARGETS = [pytest.param("cpu", torch.float32, id="cpu-fp32"),
           pytest.param("cuda", torch.float32, id="gpu-fp32", marks=_GPU),
           pytest.param("cuda", torch.bfloat16, id="gpu-bf16", marks=_GPU)]
FP32_TARGETS = TARGETS[:2]


def row_err(got, want):
    """RMS of the difference (mean over the vocabulary taken off) over the RMS of the centred reference, per row."""
    d = got.double() - want.double()
    d = d - d.mean(-1, keepdim=True)
    w = want.double() - want.double().mean(-1, keepdim=True)
    return d.pow(2).mean(-1).sqrt() / w.pow(2).mean(-1).sqrt().clamp_min(1e-9)


def rel_err(got, want):
    return row_err(got, want).max().item()


def close(got, want, dtype):
    """fp32: every row within 2e-4. bf16: rounding level - rows within 4 % on average and no row beyond 25 %; a wrong
    mechanism is off by tens of percent on most rows."""
    e = row_err(got, want)
    if dtype == torch.float32:
        return e.max().item() < 2e-4
    return e.mean().item() < 4e-2 and e.max().item() < 0.25


def make_engine(cfg, sd, device, dtype, max_tokens=512, max_seqs=4, graphs=None):
    model = LuketarModel(LuketarConfig.from_json(cfg), device=device, dtype=dtype).load_state(sd)
    from generativeaiexamples_amd.engine.tokenizer import load_tokenizer
    graphs = (device != "cpu") if graphs is None else graphs
    return LLMEngine(model, load_tokenizer(None, "llama3", cfg["vocab"]), EngineConfig(
        max_num_seqs=max_seqs, num_blocks=max_tokens // ops.BLOCK, max_model_len=max_tokens, max_batched_tokens=1 << 20,
        use_graphs=graphs, graph_batch_sizes=(1, 2, 4), decode_steps=1))


def run_schedule(eng, prompts, schedule):
    """schedule: list of steps, each a list of (request name, count). Returns {name: logits [len, vocab]} with every
    position's logits; requests end when their tokens are used up."""
    at = {n: 0 for n in prompts}
    got = {n: [] for n in prompts}
    for step in schedule:
        entries, end = [], []
        for name, count in step:
            lo = at[name]
            entries.append((name, prompts[name][lo:lo + count], list(range(count))))
            at[name] = lo + count
            if at[name] == len(prompts[name]):
                end.append(name)
        out = eng.replay_step(entries, end)
        r = 0
        for name, count in step:
            got[name].append(out[r:r + count])
            r += count
    return {n: torch.cat(v) for n, v in got.items() if v}


def tokens(n, vocab, seed):
    g = torch.Generator().manual_seed(seed)
    return torch.randint(0, vocab, (n,), generator=g).tolist()


def config_for(dtype, layers, **kw):
    """The test's configuration. An expert choice is a discrete decision: with random weights some position always has
    two router logits closer than bf16 rounding of the router's input. So bf16 runs take every expert (the same kernels,
    no decision), and the choice itself is tested in fp32 (CPU and GPU) on prompts without a near-tie (clear_tokens)."""
    if dtype == torch.bfloat16:
        layers = [l if (l["mlp"] or {}).get("kind") != "moe" else
                  dict(l, mlp=dict(l["mlp"], router=dict(l["mlp"]["router"], top=l["mlp"]["router"]["experts"])))
                  for l in layers]
    return O.make_config(layers, **kw)


def clear_tokens(n, cfg, sd, seed, gap=1e-4):
    """Random tokens whose router has no near-tie between the last chosen and the first rejected expert, and whose
    logits are well-conditioned: with few tokens seen, a matrix memory's output is about (k . q) v over its own norm, so
    a prompt with k . q near zero turns fp32 rounding of the weights alone into a visible difference."""
    g = torch.Generator().manual_seed(seed)
    sd2 = {k: v.double() * (1 + 1e-7 * torch.randn(v.shape, generator=g)) for k, v in sd.items()}
    for s in range(seed, seed + 50):
        t = tokens(n, cfg["vocab"], s)
        margins = []
        want = O.forward(cfg, sd, t, margins=margins)
        if min(margins + [math.inf]) > gap and rel_err(O.forward(cfg, sd2, t), want) < 4e-5:
            return t
    raise AssertionError("no clear-cut prompt found")


def cuts(n, sizes):
    out, i = [], 0
    while n > 0:
        c = min(n, sizes[i % len(sizes)])
        out.append(c)
        n -= c
        i += 1
    return out


FULL = [O.dense(O.mem()), O.moe(O.att()), O.no_ff(O.att(heads=2, dim=6, vdim=5, q_rank=7, kv_rank=9, scale=0.8)),
        O.again(O.moe(O.att()), 1), O.moe(O.mem(heads=2, dim=5, vdim=7, gate_cap=3.0), ff=8, experts=4, top=1, shared=0)]


# ------------------------------------------------------------------------------------------------ each mechanism alone
@pytest.mark.parametrize("device,dtype", TARGETS)
@pytest.mark.parametrize("layers,streams", [
    ([O.no_ff(O.att())], 3), ([O.no_ff(O.att(heads=1, dim=4, vdim=20, q_rank=5, kv_rank=3, scale=1.0))], 1),
    ([O.no_ff(O.att(heads=7, dim=16, vdim=8, q_rank=64, kv_rank=32, scale=0.1))], 5),
    ([O.no_ff(O.att(heads=33, dim=4, vdim=4, q_rank=8, kv_rank=64, scale=0.7))], 2),
    ([O.no_ff(O.mem())], 3), ([O.no_ff(O.mem(heads=1, dim=3, vdim=30, gate_cap=1.0))], 1),
    ([O.no_ff(O.mem(heads=5, dim=33, vdim=1, gate_cap=30.0))], 9),
    ([O.dense(O.mem())], 2), ([O.dense(O.mem(), ff=50, limit=0.3)], 4),
    ([O.moe(O.mem())], 3), ([O.moe(O.mem(), ff=20, experts=3, top=1, shared=0)], 1),
    ([O.moe(O.att(), ff=40, experts=12, top=5, limit=0.4, shared=8, shared_limit=0.2)], 2),
    ([O.moe(O.att(), experts=4, top=4)], 4),
    ([O.no_ff(O.mem()), O.again(O.no_ff(O.mem()), 0), O.again(O.no_ff(O.mem()), 1)], 2)],
    ids=["latent", "latent-1head", "latent-7heads-5streams", "latent-33heads", "mlstm", "mlstm-1head-tight-cap",
         "mlstm-5heads-9streams", "dense", "dense-tight-limit", "moe", "moe-top1-1stream", "moe-top5-tight", "moe-all-experts",
         "shared-weights"])
def test_single_mechanism(layers, streams, device, dtype):
    cfg = config_for(dtype, layers, width=48, streams=streams)
    sd = O.random_checkpoint(cfg, 1)
    toks = clear_tokens(37, cfg, sd, 2)
    want = O.forward(cfg, sd, toks)
    eng = make_engine(cfg, sd, device, dtype)
    got = run_schedule(eng, {"a": toks}, [[("a", len(toks))]])["a"]
    assert close(got, want, dtype)


@pytest.mark.parametrize("device", [pytest.param("cpu"), pytest.param("cuda", marks=_GPU)])
def test_hyper_connect_against_equations(device):
    """Closing a sublayer (mix indexed [from, to], all streams from the old ones), opening the next (layer norm without
    bias), both in one pass, from distinct streams and from the embedding output; rows on and off the grid of four, wider
    than one workgroup's registers, and 1 to 16 streams."""
    g = torch.Generator().manual_seed(0)
    rn = lambda *s: torch.randn(*s, generator=g)  # noqa: E731
    for T, ns, D in ((3, 4, 256), (600, 3, 64), (5, 2, 70), (2, 6, 4100), (4, 1, 36), (1, 3, 17000), (2, 16, 5)):
        X, y, mix, ow, iw, nw, x0 = rn(T, ns, D), rn(T, D + 3), rn(ns, ns), rn(ns), rn(ns), rn(D), rn(T, D)
        for first in (False, True):
            for close_it in (False, True):
                for open_it in (False, True):
                    if not (close_it or open_it):
                        continue
                    old = [x0.double()] * ns if first else [X[:, s].double() for s in range(ns)]
                    new = O.write_streams(old, mix.double(), ow.double(), y[:, 3:].double()) if close_it else old
                    Xd = X.clone().to(device)
                    kw = dict(y=y.to(device)[:, 3:], mix=mix.to(device), out_w=ow.to(device)) if close_it else {}
                    if open_it:
                        kw.update(in_w=iw.to(device), norm_w=nw.to(device), out_dtype=torch.float32)
                    out = ops.hyper_connect(Xd, x0.to(device) if first else None, eps=1e-5, **kw)
                    assert torch.allclose(Xd.cpu().double(), torch.stack(new, 1), atol=1e-4, rtol=1e-5)
                    if open_it:
                        want = O.layer_norm(O.read_streams(new, iw.double()), nw.double(), 1e-5)
                        assert torch.allclose(out.cpu().double(), want, atol=1e-4, rtol=1e-4)
                    else:
                        assert out is None


@pytest.mark.parametrize("device,dtype", TARGETS)
@pytest.mark.parametrize("H,dk,dv", [(3, 5, 7), (1, 70, 9), (2, 130, 36), (2, 16, 70), (2, 64, 128), (1, 24, 200)])
def test_matrix_memory_from_nonzero_states(H, dk, dv, device, dtype):
    """The matrix-memory core from states that are not zero in scattered slots - a step with portions (a chunk's edge, two
    chunks and a bit, a single token) and a step of single tokens -, gates up to the cap, long enough for the form that
    runs spans of one sequence side by side; other slots stay untouched."""
    g = torch.Generator().manual_seed(3)
    rn = lambda *s: torch.randn(*s, generator=g)  # noqa: E731
    cap, eps = 6.0, 1e-5
    dev = torch.device(device)
    for lens, slots_l in (([64, 150, 1, 7], [5, 0, 3, 2]), ([1, 1, 1], [4, 1, 2]), ([300], [3])):
        T, n = sum(lens), 2 * H * dk + 2 * H * dv
        proj, gl = (rn(T, n + 3) * 0.7).to(dtype), rn(T, 2 * H + 1) * 3
        ib, fb, nw = rn(H), rn(H) * 3 + 3, rn(H * dv)
        S, nn, m = rn(6, H, dk, dv), rn(6, H, dk), rn(6, H)
        cu_l = [0]
        for c in lens:
            cu_l.append(cu_l[-1] + c)
        i32 = lambda v: torch.tensor(v, dtype=torch.int32, device=dev)  # noqa: E731
        a, b, c = 3 + H * dk, 3 + 2 * H * dk, 3 + 2 * H * dk + H * dv
        P, G = proj.to(dev), gl.to(dev)
        Sd, nd, md = S.clone().to(dev), nn.clone().to(dev), m.clone().to(dev)
        got = ops.mlstm(P[:, 3:a], P[:, a:b], P[:, b:c], G[:, 1:1 + H], G[:, 1 + H:], ib.to(dev), fb.to(dev), cap, P[:, c:],
                        nw.to(dev), Sd, nd, md, i32(cu_l), i32(slots_l), dk ** -0.5, eps, DEN_EPS, torch.float32
                        if dtype == torch.float32 else dtype).cpu().double()
        pd = proj.double()
        li, lf = O.log_gates(gl[:, 1:1 + H].double() + ib.double(), gl[:, 1 + H:].double() + fb.double(), cap)
        tol = 2e-5 if dtype == torch.float32 else 1e-2
        for j, sl in enumerate(slots_l):
            lo, hi = cu_l[j], cu_l[j + 1]
            for h in range(H):
                q = pd[lo:hi, 3 + h * dk:3 + (h + 1) * dk] * dk ** -0.5
                o, S1, n1, m1 = O.mlstm_cell(q, pd[lo:hi, a + h * dk:a + (h + 1) * dk], pd[lo:hi, b + h * dv:b + (h + 1) * dv],
                                             li[lo:hi, h], lf[lo:hi, h], S[sl, h].double(), nn[sl, h].double(), m[sl, h].double())
                want = O.unit_rms(o, eps) * nw[h * dv:(h + 1) * dv].double() * O.sigmoid(pd[lo:hi, c + h * dv:c + (h + 1) * dv])
                err = (got[lo:hi, h * dv:(h + 1) * dv] - want).norm() / want.norm()
                assert err < tol, (lens, j, h, float(err))
                for have, ref in ((Sd[sl, h], S1), (nd[sl, h], n1)):
                    assert (have.cpu().double() - ref).norm() <= 2e-5 * ref.norm() + 1e-9, (lens, j, h)
                assert abs(float(md[sl, h]) - float(m1)) < 1e-5 * (1 + abs(float(m1)))
        for sl in set(range(6)) - set(slots_l):
            assert torch.equal(Sd[sl].cpu(), S[sl]) and torch.equal(nd[sl].cpu(), nn[sl]) and torch.equal(md[sl].cpu(), m[sl])


@pytest.mark.parametrize("device,dtype", FP32_TARGETS)
def test_small_ops_against_equations(device, dtype):
    """The router where the bias changes the choice and logits are large; per-head products with and without the gate,
    sizes on and off the matrix-core grid; both latent norms and the cache row through scattered pages; sinks that
    differ by head."""
    g = torch.Generator().manual_seed(5)
    rn = lambda *s: torch.randn(*s, generator=g)  # noqa: E731
    dev = torch.device(device)
    # router: bias inside the logits, weights from the chosen logits only (a column slice of a padded projection)
    E, k = 7, 3
    z, b = rn(50, 16) * 20, rn(E) * 30
    ids, w = ops.moe_route(z.to(dev)[:, :E], k, score="chosen", bias=b.to(dev))
    zz = z[:, :E].double() + b.double()
    top, want = zz.topk(k, -1)
    assert not torch.equal(want.sort(-1).values, z[:, :E].topk(k, -1).indices.sort(-1).values)
    assert torch.equal(ids.cpu().long(), want)
    assert torch.allclose(w.cpu().double(), torch.softmax(top, -1), atol=1e-6)
    # per-head products
    for T, H, N, K in ((3, 2, 20, 12), (70, 3, 32, 24), (130, 1, 100, 64), (5, 4, 7, 9)):
        x, W, gt = rn(T, H * K + 2), rn(H, N, K), rn(T, H * N + 1)
        want = torch.einsum("thk,hnk->thn", x[:, 2:].double().reshape(T, H, K), W.double()).reshape(T, H * N)
        assert torch.allclose(ops.head_linear(x.to(dev)[:, 2:], W.to(dev)).cpu().double(), want, atol=1e-4)
        got = ops.head_linear(x.to(dev)[:, 2:], W.to(dev), gt.to(dev)[:, 1:]).cpu().double()
        assert torch.allclose(got, want * O.sigmoid(gt[:, 1:].double()), atol=1e-4)
    # latent norms, cache rows in scattered slots
    T, RQ, R = 6, 37, 21
    both, wq, wk = rn(T, RQ + R + 1), rn(RQ), rn(R)
    both[2] *= 1e-3                                  # small rows: the epsilon inside the root matters
    kc, vc = torch.zeros(9, 1, ops.BLOCK, R, device=dev), torch.zeros(9, 1, R, ops.BLOCK, device=dev)
    slots = [5 * ops.BLOCK + 3, 7, 8, 2 * ops.BLOCK + 15, 40, 41]
    q = ops.latent_norm_write(both.to(dev)[:, :RQ], wq.to(dev), both.to(dev)[:, RQ:RQ + R], wk.to(dev),
                              torch.tensor(slots, dtype=torch.int32, device=dev), kc, vc, 1e-5).cpu().double()
    assert torch.allclose(q, O.unit_rms(both[:, :RQ].double(), 1e-5) * wq.double(), atol=1e-5)
    c = O.unit_rms(both[:, RQ:RQ + R].double(), 1e-5) * wk.double()
    for t, s in enumerate(slots):
        assert torch.allclose(kc[s // ops.BLOCK, 0, s % ops.BLOCK].cpu().double(), c[t], atol=1e-5)
        assert torch.allclose(vc[s // ops.BLOCK, 0, :, s % ops.BLOCK].cpu().double(), c[t], atol=1e-5)
    assert (kc.cpu() != 0).any(-1).sum() == T


# ------------------------------------------------------------------------------------ whole model, schedules, batches
@pytest.mark.parametrize("device,dtype", TARGETS)
def test_prefill_decode_portions(device, dtype):
    """Whole prompt, token-by-token decoding from the first token on, and portions of 2 / 3 / 5 / 17 / 1 tokens: every
    position's logits equal the oracle's, so they do not depend on how the prompt was cut. The sum of the streams after
    every layer equals the oracle's."""
    cfg = config_for(dtype, FULL)
    sd = O.random_checkpoint(cfg, 3)
    toks = clear_tokens(61, cfg, sd, 4)
    res = []
    want = O.forward(cfg, sd, toks, res)
    eng = make_engine(cfg, sd, device, dtype)
    for name, sizes in (("whole", [61]), ("decode", [1]), ("prefill+decode", [30] + [1] * 31), ("small", [2, 3, 5, 17, 1]),
                        ("twos", [2])):
        sched = [[(name, c)] for c in cuts(61, sizes)]
        got = run_schedule(eng, {name: toks}, sched)[name]
        assert close(got, want, dtype), name
    eng.model.capture_residuals = []
    run_schedule(eng, {"r": toks}, [[("r", 61)]])
    got_res, eng.model.capture_residuals = eng.model.capture_residuals, None
    assert len(got_res) == len(res)
    for i, (gr, wr) in enumerate(zip(got_res, res)):
        e = (gr.cpu().double() - wr).norm() / wr.norm()
        assert e < (1e-5 if dtype == torch.float32 else 6e-2), (i, float(e))


@pytest.mark.parametrize("device,dtype", TARGETS)
def test_mixed_batches_and_reuse(device, dtype):
    """Unequal requests in one batch (portions beside single tokens) against each alone; a pool of two state slots and
    few pages, so slots and pages of finished requests are used again by later ones."""
    cfg = config_for(dtype, FULL)
    sd = O.random_checkpoint(cfg, 5)
    lens = dict(a=45, b=18, c=33, d=1, e=26)
    prompts = {n: clear_tokens(L, cfg, sd, 10 + 50 * i) for i, (n, L) in enumerate(lens.items())}
    want = {n: O.forward(cfg, sd, t) for n, t in prompts.items()}
    eng = make_engine(cfg, sd, device, dtype, max_tokens=96, max_seqs=2)
    sched = [[("a", 20), ("b", 3)], [("a", 1), ("b", 15)],          # b ends: its slot and pages go back
             [("a", 1), ("c", 2)], [("c", 17), ("a", 5)], [("a", 1), ("c", 1)], [("a", 17), ("c", 13)],  # a, c end
             [("d", 1), ("e", 7)], [("e", 2)], [("e", 1)], [("e", 16)]]
    got = run_schedule(eng, prompts, sched)
    for n in prompts:
        assert close(got[n], want[n], dtype), n
    assert eng.sched.num_free_blocks() == 96 // ops.BLOCK and not eng.model.pool.slot_of


@pytest.mark.parametrize("device,dtype", TARGETS)
def test_first_tokens_and_long_decode(device, dtype):
    """Positions 0..4 of a sequence (zero states with the maximum at zero, one key beside the sink) and 150 single-token
    steps across many page borders."""
    cfg = config_for(dtype, [O.moe(O.att()), O.no_ff(O.mem()), O.dense(O.att(heads=2, kv_rank=16, q_rank=8))])
    sd = O.random_checkpoint(cfg, 7)
    toks = clear_tokens(155, cfg, sd, 8)
    want = O.forward(cfg, sd, toks)
    eng = make_engine(cfg, sd, device, dtype)
    got = run_schedule(eng, {"a": toks}, [[("a", 1)] for _ in toks])["a"]
    assert close(got[:5], want[:5], dtype)
    assert close(got, want, dtype)


@pytest.mark.parametrize("device,dtype", FP32_TARGETS)
def test_far_token_through_state(device, dtype):
    """Slowly forgetting matrix memory and no attention: changing four tokens 300 positions back changes the last logits
    (oracle), and the framework follows it, through a prompt cut at odd places and single-token steps."""
    cfg = O.make_config([O.no_ff(O.mem(heads=2, dim=4, vdim=4)), O.no_ff(O.mem(heads=1, dim=6, vdim=4))], width=32, vocab=64)
    sd = O.random_checkpoint(cfg, 9, slow_forget=True)
    a = clear_tokens(320, cfg, sd, 11)
    b = list(a)
    for i in (5, 6, 7, 8):
        b[i] = (b[i] + 13) % cfg["vocab"]
    wa, wb = O.forward(cfg, sd, a)[-1:], O.forward(cfg, sd, b)[-1:]
    assert rel_err(wb, wa) > 2e-3  # the far tokens matter
    eng = make_engine(cfg, sd, device, dtype)
    sched = lambda n: [[(n, c)] for c in cuts(320, [33, 2, 64, 1, 100])]  # noqa: E731
    got = run_schedule(eng, {"a": a, "b": b}, sched("a") + sched("b"))
    assert rel_err(got["a"][-1:], wa) < 2e-4 and rel_err(got["b"][-1:], wb) < 2e-4


def _latent_probe(device, dtype, n_ctx, hot, portion, R=8, query=-1, H=2, score=30.0, sink=None):
    """ops-level: latents of n_ctx positions through the paged cache (pages deliberately scattered). Every latent is
    orthogonal to one probing direction except the one at position `hot`, which lies along it (length sqrt(R) after its
    norm); the query at `query` points along it so that its score is `score`. The softmax puts all its weight on the hot
    key when that key is visible. Returns the component of that query's output along the direction over sqrt(R): about 1
    if the key was seen, about 0 if not."""
    B = ops.BLOCK
    dev = torch.device(device)
    nb = (n_ctx + B - 1) // B
    pages = list(range(nb + 3))[::-1][:nb]  # not the identity
    kc = torch.zeros(nb + 4, 1, B, R, dtype=dtype, device=dev)
    vc = torch.zeros(nb + 4, 1, R, B, dtype=dtype, device=dev)
    g = torch.Generator().manual_seed(0)
    qi = query % n_ctx
    d = torch.randn(R, generator=g)
    d = d / d.norm()
    lat = torch.randn(n_ctx, R, generator=g)
    lat = lat - (lat @ d)[:, None] * d
    lat[hot] = d
    q = torch.randn(n_ctx, H, R, generator=g) * 0.1
    q[qi] = d * score / R ** 0.5
    sinks = torch.full((H,), -1e4) if sink is None else torch.tensor(sink)
    one = torch.ones(R, device=dev)
    bt = torch.tensor([pages], dtype=torch.int32, device=dev)
    done, res = 0, None
    for c in cuts(n_ctx, portion):
        pos = torch.arange(done, done + c)
        slots = torch.tensor([pages[p // B] * B + p % B for p in pos.tolist()], dtype=torch.int32, device=dev)
        x = lat[pos].to(dev, dtype)
        ops.latent_norm_write(x, one, x, one, slots, kc, vc, 1e-6)
        out = ops.window_attention(q[pos].reshape(c, H * R).to(dev, dtype), kc, vc, bt,
                                   torch.tensor([0, c], dtype=torch.int32, device=dev),
                                   torch.tensor([done + c], dtype=torch.int32, device=dev), H, 1, R, R, 1.0,
                                   sink=sinks.to(dev))
        if done <= qi < done + c:
            res = out[qi - done].float().cpu().view(H, R)
        done += c
    return (res @ d / R ** 0.5).tolist()


PORTIONS = {"prompt": [1000], "decode": [1], "portions": [7, 2, 30]}


@pytest.mark.parametrize("device,dtype", FP32_TARGETS)
@pytest.mark.parametrize("portion", PORTIONS.values(), ids=PORTIONS.keys())
def test_far_keys_page_borders_causal_edge_and_sinks(device, dtype, portion):
    """One key among hundreds carries the output: at position 0, at page borders, far away, the query's own position
    (seen) and the one after it (not seen); in prompts, in portions and in single-token steps. Sinks differ by head: a
    visible hot key of score x against a sink of score s gets the weight 1 / (1 + e^(s - x))."""
    n = 340
    por = portion if portion != [1] else [300, 1]
    for hot in (0, 1, 15, 16, 17, 31, 32, 63, 64, 200, n - 2, n - 1):
        out = _latent_probe(device, dtype, n, hot, por)
        assert all(abs(o - 1.0) < 2e-3 for o in out), (hot, out)
    for qi in (0, 5, 15, 16, 31, 32, 40, 63, 64):   # causal edge: own position in, next position out
        assert all(abs(o - 1.0) < 2e-3 for o in _latent_probe(device, dtype, 70, qi, portion, query=qi)), qi
        assert all(abs(o) < 2e-3 for o in _latent_probe(device, dtype, 70, qi + 1, portion, query=qi)), qi
    out = _latent_probe(device, dtype, 1, 0, [1], score=1.0, sink=[1.0, 1.0 + math.log(3.0)])
    assert abs(out[0] - 0.5) < 2e-3 and abs(out[1] - 0.25) < 2e-3, out
    out = _latent_probe(device, dtype, n, 33, por, score=30.0, sink=[30.0, -50.0])
    assert abs(out[0] - 0.5) < 2e-3 and abs(out[1] - 1.0) < 2e-3, out
    out = _latent_probe(device, dtype, n, 33, por, score=30.0, sink=[80.0, 30.0 + math.log(3.0)])
    assert abs(out[0]) < 2e-3 and abs(out[1] - 0.25) < 2e-3, out


@_GPU
@pytest.mark.parametrize("R,H", [(32, 4), (64, 3), (96, 8), (128, 16), (160, 2), (192, 5), (256, 16), (48, 40), (256, 1),
                                 (128, 33), (512, 4)])
def test_far_keys_bf16_kernels(R, H):
    """The same stand-out key probes in bf16: latent sizes and head counts that take the matrix-core kernels beside sizes
    off their grid, in prompts, portions and single-token steps; sinks per head."""
    n, dt = 700, torch.bfloat16
    sink = [30.0 if h % 2 else -50.0 for h in range(H)]
    for portion in ([1000], [170, 140, 9, 11], [220, 3, 107], [699, 1]):
        for hot in (0, 15, 16, 31, 32, 333, n - 2, n - 1):
            out = _latent_probe("cuda", dt, n, hot, portion, R, H=H)
            assert all(abs(o - 1.0) < 0.05 for o in out), (portion, hot, out)
        out = _latent_probe("cuda", dt, n, 64, portion, R, H=H, sink=sink)
        assert all(abs(o - (0.5 if h % 2 else 1.0)) < 0.06 for h, o in enumerate(out)), (portion, out)
        for qi in (0, 7, 31, 32, 100, 149):
            assert all(abs(o - 1.0) < 0.05 for o in _latent_probe("cuda", dt, 151, qi, portion, R, H=H, query=qi)), qi
            assert all(abs(o) < 0.05 for o in _latent_probe("cuda", dt, 151, qi + 1, portion, R, H=H, query=qi)), qi


@_GPU
@pytest.mark.parametrize("R,H", [(64, 16), (128, 8), (256, 16), (96, 6)])
def test_latent_attention_bf16_against_reference(R, H):
    """Unequal requests in one step - prompts, a continued portion, single tokens - through the bf16 kernels against the
    fp32 reference of the same op on the same (bf16-rounded) values; then a step of single tokens only."""
    g = torch.Generator().manual_seed(1)
    rn = lambda *s: torch.randn(*s, generator=g)  # noqa: E731
    B = ops.BLOCK
    for ctx, qlen in (([300, 77, 513, 40], [300, 20, 1, 1]), ([300, 77, 1, 1025], [1, 1, 1, 1]), ([90], [64])):
        S = len(ctx)
        nb = [(c + B - 1) // B for c in ctx]
        perm = torch.randperm(sum(nb) + 2, generator=g).tolist()
        bt = torch.zeros(S, max(nb), dtype=torch.int32)
        for s in range(S):
            bt[s, :nb[s]] = torch.tensor(perm[sum(nb[:s]):sum(nb[:s + 1])], dtype=torch.int32)
        kc = rn(sum(nb) + 2, 1, B, R).to(torch.bfloat16)
        vc = kc.transpose(2, 3).contiguous()
        T = sum(qlen)
        q = (rn(T, H * R) * 2 * R ** -0.5).to(torch.bfloat16)
        sink = rn(H) * 2
        cu = torch.tensor([sum(qlen[:s]) for s in range(S + 1)], dtype=torch.int32)
        args = (bt, cu, torch.tensor(ctx, dtype=torch.int32))
        want = ops.window_attention(q.float(), kc.float(), vc.float(), *args, H, 1, R, R, 0.9, sink=sink)
        got = ops.window_attention(q.cuda(), kc.cuda(), vc.cuda(), *[a.cuda() for a in args], H, 1, R, R, 0.9,
                                   sink=sink.cuda()).float().cpu()
        e = (got - want).norm(dim=-1) / want.norm(dim=-1)
        assert e.max() < 8e-3, (ctx, float(e.max()), int(e.argmax()))


@_GPU
@pytest.mark.parametrize("act", [None, "relu2", "swiglu", "clamp_glu"])
@pytest.mark.parametrize("T,E,k,N,K", [(1, 8, 2, 96, 192), (7, 4, 2, 64, 320), (30, 6, 2, 160, 64), (60, 8, 3, 32, 1408)])
def test_decode_sized_expert_products(T, E, k, N, K, act):
    """Grouped expert products of a few rows whose K is off the staged weight stream's grid: some experts without rows, one
    with most of them, every activation, against fp32 products of the same bf16 values."""
    g = torch.Generator().manual_seed(2)
    rn = lambda *s: torch.randn(*s, generator=g)  # noqa: E731
    x, W = rn(T, K).to(torch.bfloat16), (rn(E, N, K) * K ** -0.5).to(torch.bfloat16)
    ids = torch.stack([torch.randperm(E - 1, generator=g)[:k] for _ in range(T)]).int()     # the last expert gets none
    ids[:, 0] = torch.where(torch.rand(T, generator=g) < 0.7, torch.zeros(T), ids[:, 0].float()).int()
    rows, offs, _ = ops.moe_dispatch(ids.cuda(), E)
    for gather in (True, False):
        a = x if gather else x[rows.cpu().long()]
        got = ops.moe_gemm(a.cuda(), rows if gather else None, W.cuda(), offs, T * k, act=act, act_param=0.7).float().cpu()
        want = ops.moe_gemm(a.float(), rows.cpu() if gather else None, W.float(), offs.cpu(), T * k, act=act, act_param=0.7)
        assert (got - want).norm() < 6e-3 * want.norm() and (got - want).abs().max() < 0.05 * want.abs().max()


@_GPU
def test_matrix_core_kernels_in_model():
    """bf16 model with sizes on the matrix-core grids: portions take the matrix-core kernels, single tokens the
    decode kernels; both against the oracle, alone and in a mixed batch."""
    layers = [O.moe(O.att(heads=8, dim=32, vdim=48, q_rank=64, kv_rank=128, scale=0.2), ff=64, experts=4, shared=64),
              O.dense(O.mem(heads=4, dim=32, vdim=64), ff=192),
              O.moe(O.att(heads=4, dim=16, vdim=64, q_rank=128, kv_rank=64, scale=0.25), ff=128, experts=4, shared=0)]
    cfg = config_for(torch.bfloat16, layers, width=128, vocab=128, streams=2)
    sd = O.random_checkpoint(cfg, 61)
    prompts = {"a": tokens(150, 128, 62), "b": tokens(90, 128, 163)}
    want = {n: O.forward(cfg, sd, t) for n, t in prompts.items()}
    eng = make_engine(cfg, sd, "cuda", torch.bfloat16)
    got = run_schedule(eng, prompts, [[("a", 150)], [("b", 40)], [("b", 3)], [("b", 47)]])
    for n in prompts:
        assert close(got[n], want[n], torch.bfloat16), n
    got = run_schedule(eng, prompts, [[("a", 100), ("b", 5)], [("a", 1), ("b", 60)], [("a", 1), ("b", 1)], [("a", 48), ("b", 24)]])
    for n in prompts:
        assert close(got[n], want[n], torch.bfloat16), n


@_GPU
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16], ids=["fp32", "bf16"])
def test_long_prompt_against_oracle(dtype):
    """A prompt long enough for the span-parallel matrix memory, whole and cut in two, against the oracle."""
    cfg = config_for(dtype, [O.moe(O.mem(heads=2, dim=16, vdim=16)), O.no_ff(O.att()), O.no_ff(O.mem(heads=1, dim=20, vdim=150))])
    sd = O.random_checkpoint(cfg, 41)
    toks = clear_tokens(640, cfg, sd, 42, gap=3e-5)
    want = O.forward(cfg, sd, toks)
    eng = make_engine(cfg, sd, "cuda", dtype, max_tokens=1024)
    for name, sizes in (("whole", [640]), ("two", [530, 110])):
        got = run_schedule(eng, {name: toks}, [[(name, c)] for c in sizes])[name]
        assert close(got, want, dtype), name


@pytest.mark.parametrize("device,dtype", TARGETS)
@pytest.mark.parametrize("shape", ["wide-odd", "tiny", "one-stream-unit-scale"])
def test_other_shapes(shape, device, dtype):
    kw = {}
    if shape == "wide-odd":
        layers = [O.moe(O.att(heads=6, dim=12, vdim=20, q_rank=30, kv_rank=50, scale=0.3), ff=48, experts=9, top=3, shared=40),
                  O.no_ff(O.mem(heads=4, dim=24, vdim=10)), O.dense(O.att(kv_rank=8, q_rank=40), ff=100)]
        kw = dict(width=72, vocab=201, streams=6, eps=1e-3)
    elif shape == "tiny":
        layers = [O.moe(O.mem(heads=1, dim=1, vdim=2), ff=4, experts=2, top=1, shared=2),
                  O.no_ff(O.att(heads=1, dim=1, vdim=1, q_rank=1, kv_rank=2))]
        kw = dict(width=8, vocab=20, streams=2)
    else:
        layers, kw = FULL[:2], dict(width=24, streams=1, scale=1.0)
    cfg = config_for(dtype, layers, **kw)
    sd = O.random_checkpoint(cfg, 23)
    toks = clear_tokens(50, cfg, sd, 22)
    want = O.forward(cfg, sd, toks)
    eng = make_engine(cfg, sd, device, dtype)
    got = run_schedule(eng, {"a": toks}, [[("a", c)] for c in cuts(50, [19, 1, 1, 6])])["a"]
    assert close(got, want, dtype)


# -------------------------------------------------------------------------- entry points: registry, generation, runner
def _write_checkpoint(path, cfg, sd):
    from safetensors.torch import save_file
    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(cfg, f)
    save_file({k: v.to(torch.bfloat16).contiguous() for k, v in sd.items()}, os.path.join(path, "model.safetensors"))


@pytest.mark.parametrize("device,dtype", FP32_TARGETS)
def test_greedy_generation_through_engine(tmp_path, device, dtype):
    """A checkpoint directory -> registry -> LLMEngine.generate (its scheduler, cache, state slots, sampling): greedy
    continuations of three prompts served together equal the oracle's argmax continuation, token by token."""
    cfg = O.make_config(FULL[:4], width=32, vocab=96)
    sd = O.random_checkpoint(cfg, 31)
    _write_checkpoint(str(tmp_path / "m"), cfg, sd)
    model, tok, _ = build_llm(weights=str(tmp_path / "m"), device=device, dtype=dtype)
    assert isinstance(model, LuketarModel)
    eng = LLMEngine(model, tok, EngineConfig(max_num_seqs=4, num_blocks=32, max_model_len=256, prefill_chunk=16,
                                             max_batched_tokens=24, use_graphs=device != "cpu",
                                             graph_batch_sizes=(1, 2, 4), decode_steps=1))
    prompts = [tokens(n, 96, 40 + n) for n in (9, 23, 2)]
    outs = eng.generate(prompts, SamplingParams(max_tokens=12, temperature=0.0, ignore_eos=True))
    for p, o in zip(prompts, outs):
        assert len(o.output_ids) == 12
        seq = list(p)
        for t in o.output_ids:
            row = O.forward(cfg, sd, seq)[-1]     # the oracle's argmax, up to a near-tie of its top logits
            assert row[t] >= row.max() - 1e-3 * (row.max() - row.min()), (len(seq), t, int(row.argmax()))
            seq.append(int(t))


def test_preset_and_generation_cpu():
    model, tok, name = build_llm("tiny-luketar", device="cpu", dtype=torch.float32)
    assert name == "tiny-luketar" and isinstance(model, LuketarModel)
    eng = LLMEngine(model, tok, EngineConfig(max_num_seqs=2, num_blocks=16, max_model_len=128, use_graphs=False))
    outs = eng.generate([[1, 2, 3], [4, 5]], SamplingParams(max_tokens=5, temperature=0.0, ignore_eos=True))
    assert [len(o.output_ids) for o in outs] == [5, 5]


@pytest.mark.parametrize("device", [pytest.param("cpu", id="cpu"), pytest.param("cuda:0", id="gpu", marks=_GPU)])
def test_runner_script(tmp_path, device):
    """The replay script: steps on stdin, logits files out, slots and pages reused within a pool made for the live
    requests only."""
    cfg = O.make_config(FULL[:3], width=32, vocab=96)
    sd = O.random_checkpoint(cfg, 33)
    _write_checkpoint(str(tmp_path / "m"), cfg, sd)
    a, b = tokens(40, 96, 1), tokens(21, 96, 2)
    wa, wb = O.forward(cfg, sd, a), O.forward(cfg, sd, b)
    steps = [dict(step=0, entries=[dict(id="a", tokens=a[:30], want=[0, 29])], end=[]),
             dict(step=1, entries=[dict(id="a", tokens=a[30:31], want=[0]), dict(id="b", tokens=b[:20], want=[19])], end=[]),
             dict(step=2, entries=[dict(id="b", tokens=b[20:], want=[])], end=["b"]),
             dict(step=3, entries=[dict(id="a", tokens=a[31:], want=[8])], end=["a"]),
             dict(step=4, entries=[dict(id="c", tokens=b, want=[20])], end=["c"])]
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    out = tmp_path / "out"
    p = subprocess.run([sys.executable, os.path.join(root, "bin", "trace_run"), "--model", str(tmp_path / "m"), "--dtype",
                        "float32", "--out", str(out), "--max-tokens", "128", "--device", device],
                       input="\n".join(json.dumps(s) for s in steps) + "\n", capture_output=True, text=True, timeout=600)
    assert p.returncode == 0, p.stderr[-2000:]
    assert [l for l in p.stdout.splitlines() if l.startswith("done")] == [f"done {i}" for i in range(5)]
    import numpy as np
    rd = lambda i: torch.from_numpy(np.fromfile(str(out / f"{i}.f32"), dtype="<f4").reshape(-1, 96))  # noqa: E731
    assert rel_err(rd(0), wa[[0, 29]]) < 2e-4 and rel_err(rd(1), torch.stack([wa[30], wb[19]])) < 2e-4
    assert not (out / "2.f32").exists()
    assert rel_err(rd(3), wa[39:40]) < 2e-4 and rel_err(rd(4), wb[20:21]) < 2e-4


def test_config_errors():
    base = O.make_config(FULL)

    def bad(edit):
        c = json.loads(json.dumps(base))
        edit(c)
        with pytest.raises(ValueError):
            LuketarConfig.from_json(c)

    bad(lambda c: c["layers"][0].update(type="conv"))
    bad(lambda c: c["layers"][0]["mlp"].update(kind="sparse"))
    bad(lambda c: c["layers"][1]["mlp"]["router"].update(top=7))     # more than there are experts
    bad(lambda c: c["layers"][3].update(weights_of=3))               # itself
    bad(lambda c: c["layers"][3].update(weights_of=9))               # no such layer
    bad(lambda c: c["layers"][3].update(weights_of=0))               # a layer of another kind
    bad(lambda c: c["layers"][3]["mixer"].update(heads=2))           # other sizes than the layer it borrows from
    bad(lambda c: c.update(streams=0))
    with pytest.raises(ValueError):
        ops.moe_route(torch.zeros(2, 6), 2, score="best")
