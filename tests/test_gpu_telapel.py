"""Telapel on the GPU against the plain implementation (tests/plain_telapel.py): each new kernel alone (the diagonal
recurrence in its four forms; the short convolution that keeps its own inputs; slopes by distance behind a cap, with
a window and a constant sink, in every attention kernel; query temperature and interleaved rotation; the
latents' preparation; softmax scores and groups by their best in the router; the clamped unit; the norm behind a
sublayer that hands the residual on as it is); whole prompts against token-by-token decoding, portions down to two
tokens and mixed batches with pages, request slots and states used again, steps that want no logits, in 32-bit and
bfloat16; long decoding; configurations drawn at random; greedy generation through LLMEngine."""

import json
import math
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

import helpers
import plain_telapel as P
import telapel_cases as cases
from mini_gpt_inference_amd import EngineConfig, SamplingParams
from mini_gpt_inference_amd.engine.llm_engine import LLMEngine
from mini_gpt_inference_amd.engine.replay import TraceReplayer
from mini_gpt_inference_amd.ops import kernels

pytestmark = pytest.mark.gpu
DEV = "cuda"
TDT = {"float32": torch.float32, "bfloat16": torch.bfloat16}


def _rnd(g, *shape, dtype="float32", scale=1.0):
    return (torch.randn(*shape, generator=g) * scale).to(TDT[dtype])


def _d(t):
    return t.to(P.DTYPE)


def _i32(x):
    return torch.tensor(x, dtype=torch.int32, device=DEV)


# Steps of a kernel-level schedule: lists of (request, first token of the request, count).  Request r's tokens
# are rows starts[r] .. of the test's arrays; its slot is r + 1 (slot 0 and the last stay untouched).
STARTS, COUNTS = [0, 140, 141, 205], [140, 1, 64, 65]
N_ROWS = 270
WHOLE = [[(0, 0, 140), (1, 0, 1), (2, 0, 64), (3, 0, 65)]]
PORTIONS = [[(0, 0, 63), (3, 0, 2)], [(0, 63, 2), (1, 0, 1), (3, 2, 62)], [(3, 64, 1), (0, 65, 74), (2, 0, 33)], [(0, 139, 1), (2, 33, 31)]]
ONE_BY_ONE = [[(r, t, 1) for r, n in enumerate(COUNTS) if t < n] for t in range(140)]


def _step_arrays(step, empty=True):
    rows, cu, pos, req, slots = [], [0], [], [], []
    for i, (r, first, count) in enumerate(step):
        rows += list(range(STARTS[r] + first, STARTS[r] + first + count))
        pos += list(range(first, first + count))
        req += [i] * count
        cu.append(len(rows))
        slots.append(r + 1)
    # a request of the padding behind the real ones: no tokens, no slot
    cu.append(len(rows))
    slots.append(-1)
    return rows, _i32(cu), _i32(pos), _i32(req), _i32(slots)


# ---------------------------------------------------------------- the diagonal recurrence
def _diagonal_case(B, S, J, dtype, seed, kind="plain"):
    """Rows [x | pad | y] as the mixer lays them out, the tensors, and the plain result for the four requests.  kind
    "slow": decays so near 1 that the first tokens are still there at the end; "fast": in places a token forgets all."""
    g = torch.Generator().manual_seed(seed)
    C = B * S
    y_off = -(-C // 16) * 16
    z = _rnd(g, N_ROWS, y_off + C + 16, dtype=dtype)
    t = {"conv": _rnd(g, C, J), "conv.b": _rnd(g, C, scale=0.3), "ra": _rnd(g, B, S, S, dtype=dtype, scale=S ** -0.5),
         "ri": _rnd(g, B, S, S, dtype=dtype, scale=S ** -0.5), "ra.b": _rnd(g, B, S), "ri.b": _rnd(g, B, S), "lam": _rnd(g, C) - 2.0}
    if kind == "slow":
        t["lam"] -= 7.0
    if kind == "fast":
        t["lam"] += torch.where(torch.rand(C, generator=g) < 0.5, 12.0, 0.0)
    want = torch.zeros(N_ROWS, C, dtype=P.DTYPE)
    for s, c in zip(STARTS, COUNTS):
        P.ROUNDING = TDT[dtype] if dtype == "bfloat16" else None
        try:
            u = P._r(P.short_conv(_d(z[s:s + c, :C]), _d(t["conv"].to(TDT[dtype])) if dtype == "bfloat16" else _d(t["conv"]), _d(t["conv.b"])))
        finally:
            P.ROUNDING = None
        r, i = (P.sigmoid(P.block_product(u, _d(t["r" + n]), _d(t["r" + n + ".b"]))) for n in ("a", "i"))
        want[s:s + c] = P.gated_recurrence(u, r, i, _d(t["lam"])) * P.gelu_tanh(_d(z[s:s + c, y_off:y_off + C]))
    if dtype == "bfloat16":
        t["conv"] = t["conv"].to(TDT[dtype]).float()
    decay = (-8.0 * P.softplus(_d(t["lam"]))).float().to(DEV)
    return z, y_off, {n: v.to(DEV) for n, v in t.items()}, decay, want


def _run_diagonal(plan, fused, B, S, J, case, pool):
    z, y_off, t, decay, _ = case
    C = B * S
    got = torch.zeros(N_ROWS, C, dtype=P.DTYPE)
    rb, ib = t["ra.b"].reshape(-1).contiguous(), t["ri.b"].reshape(-1).contiguous()
    both = torch.cat([t["ra"], t["ri"]], dim=1).contiguous()
    for step in plan:
        rows, cu, pos, req, slots = _step_arrays(step)
        n, n_req = len(rows), len(step) + 1
        single = max(c for _, _, c in step) == 1
        zs = z[rows].to(DEV)
        out = torch.full((n + 1, C + 8 if C % 8 == 0 else C), 9.0, device=DEV, dtype=z.dtype)
        kept = pool[:, C:] if J > 1 else None
        packed = kernels.pack_diagonal_gates(t["ra"], t["ri"]) if fused else None
        args = (rb, ib, decay)
        common = (slots, cu, pos, n_req, n)
        u = torch.full((n, C), 7.0, device=DEV, dtype=z.dtype)
        if fused and not single:
            scratch = torch.full((kernels.diagonal_fused_scratch_floats(n, C),), float("nan"), device=DEV)
            assert kernels.diagonal_state_fused(zs, y_off, t["conv"].t().contiguous(), t["conv.b"], packed, S, *args, pool, *common, out,
                                                scratch=scratch)
        else:
            kernels.short_conv(zs, 0, t["conv"], t["conv.b"], kept, slots, cu, req, pos, n_req, u, 0, n, single=single)
            if fused:
                assert kernels.diagonal_state_fused(zs, y_off, t["conv"].t().contiguous(), t["conv.b"], packed, S, *args, pool, *common,
                                                    out, u=u)
            else:
                gates = torch.full((n, 2 * C), 7.0, device=DEV, dtype=z.dtype)
                kernels.heads_linear(u, both, gates, n)
                scratch = None if single else torch.full((kernels.diagonal_scratch_floats(n, n_req, C),), float("nan"), device=DEV)
                kernels.diagonal_state(u, gates, *args, S, pool[:, :C], *common, out, y=zs[:, y_off:y_off + C], scratch=scratch)
        assert (out[n] == 9.0).all() and (out[:, C:] == 9.0).all()
        got[rows] = out[:n, :C].cpu().to(P.DTYPE)
    return got


@pytest.mark.parametrize("dtype,fused", [("float32", False), ("bfloat16", False), ("bfloat16", True)])
@pytest.mark.parametrize("B,S,J,kind", [
    (1, 16, 4, "plain"), (3, 48, 1, "plain"), (2, 144, 3, "plain"), (2, 64, 2, "slow"), (4, 32, 9, "fast"), (1, 272, 4, "plain"),
    (1, 512, 5, "slow"), (5, 12, 3, "plain"), (2, 7, 6, "fast")])
def test_diagonal_recurrence(dtype, fused, B, S, J, kind):
    """Whole requests of 140, 1, 64 and 65 tokens, the same in portions whose cuts fall inside, at and one token
    beside a chunk's border, and one token a step, every form of the kernels; states start as NaN and are compared too, and
    the forms go on from one another's states."""
    if fused and S % 16:
        assert kernels.pack_diagonal_gates(torch.zeros(B, S, S, dtype=torch.bfloat16), torch.zeros(B, S, S, dtype=torch.bfloat16)) is None
        return
    case = _diagonal_case(B, S, J, dtype, B * S + J, kind)
    want, C = case[4], B * S
    states = {}
    for name, plan in (("whole", WHOLE), ("portions", PORTIONS), ("one by one", ONE_BY_ONE)):
        pool = torch.full((6, J * C), float("nan"), device=DEV)
        helpers.assert_close(_run_diagonal(plan, fused, B, S, J, case, pool), want, dtype, name)
        assert torch.isnan(pool[0]).all() and torch.isnan(pool[5]).all() and torch.isfinite(pool[1:5, :C]).all()
        states[name] = pool[1:5].cpu()
    for name, st in states.items():
        helpers.assert_close(st[:, :C], states["whole"][:, :C], dtype if not fused else "float32", f"state {name}")
        long = [0, 2, 3]      # (a request of one token leaves inputs before position 0 as they were)
        assert torch.equal(st[long, C:], states["whole"][long, C:]), name
    # prompt portions by one form, single tokens by the other
    pool = torch.full((6, J * C), float("nan"), device=DEV)
    head = [[(0, 0, 101), (2, 0, 40), (3, 0, 64)]]
    tail = [[(r, t, 1) for r, first, n in ((0, 101, 140), (1, 0, 1), (2, 40, 64), (3, 64, 65)) if first <= t < n] for t in range(140)]
    other = fused if dtype == "float32" or S % 16 else not fused
    got = _run_diagonal(head, fused, B, S, J, case, pool)
    got2 = _run_diagonal([s for s in tail if s], other, B, S, J, case, pool)
    done = torch.zeros(N_ROWS, dtype=torch.bool)
    for r, n in ((0, 101), (2, 40), (3, 64)):
        done[STARTS[r]:STARTS[r] + n] = True
    helpers.assert_close(got[done], want[done], dtype, "portions")
    helpers.assert_close(got2[~done], want[~done], dtype, "single tokens behind them")


def test_many_single_tokens_in_one_step():
    """More requests than one tile of the single-token kernel, slots in any order, one of them of the padding."""
    B, S, J, n = 2, 48, 3, 39
    g = torch.Generator().manual_seed(9)
    C = B * S
    z, u = _rnd(g, n, 2 * C, dtype="bfloat16"), _rnd(g, n, C, dtype="bfloat16")
    ra, ri = (_rnd(g, B, S, S, dtype="bfloat16", scale=S ** -0.5) for _ in range(2))
    rb, ib, lam = _rnd(g, C), _rnd(g, C), _rnd(g, C) - 1.0
    pool = _rnd(g, n + 2, J * C)
    slots = torch.randperm(n + 2, generator=g)[:n].to(torch.int32)
    slots[5] = -1
    pos = [0 if t % 7 == 0 else t for t in range(n)]
    r, i = (P.sigmoid(P.block_product(_d(u), _d(w), _d(b).view(B, S))) for w, b in ((ra, rb), (ri, ib)))
    a = torch.exp(-8.0 * r * P.softplus(_d(lam)))
    before = torch.where(torch.tensor(pos)[:, None] == 0, torch.zeros(1, dtype=P.DTYPE), _d(pool[slots.clamp(min=0).long(), :C]))
    S_new = a * before + torch.sqrt(1 - a * a) * i * _d(u)
    want = S_new * P.gelu_tanh(_d(z[:, C:]))
    dev = pool.to(DEV)
    out = torch.full((n, C), 9.0, dtype=torch.bfloat16, device=DEV)
    assert kernels.diagonal_state_fused(z.to(DEV), C, torch.zeros(J, C, device=DEV), torch.zeros(C, device=DEV),
                                        kernels.pack_diagonal_gates(ra, ri).to(DEV), S, rb.to(DEV), ib.to(DEV),
                                        (-8.0 * P.softplus(_d(lam))).float().to(DEV), dev, slots.to(DEV), _i32(list(range(n + 1))), _i32(pos),
                                        n, n, out, u=u.to(DEV))
    live = slots >= 0
    helpers.assert_close(out.cpu()[live], want[live], "bfloat16", "outputs")
    assert (out.cpu()[~live] == 9.0).all()
    helpers.assert_close(dev.cpu()[slots[live].long(), :C], S_new[live], "float32", "states")
    untouched = [k for k in range(n + 2) if k not in slots.tolist()]
    assert torch.equal(dev.cpu()[untouched], pool[untouched]) and torch.equal(dev.cpu()[:, C:], pool[:, C:])


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_an_input_far_back_matters(dtype):
    """With decays near one the first token's input is still in the output after 400 tokens (a lost or restarted state
    shows), in one portion, in portions and with the last tokens one by one."""
    B, S, J = 1, 32, 2
    C, T = 32, 400
    g = torch.Generator().manual_seed(4)
    z = _rnd(g, T, 2 * C, dtype=dtype, scale=0.1)
    z[0, :C] *= 300.0
    z[:, C:] = 2.0
    zeros, one = torch.zeros(B, S, S, dtype=TDT[dtype], device=DEV), torch.zeros(C, device=DEV)
    conv = torch.tensor([[0.0, 1.0]]).repeat(C, 1).to(DEV)
    decay = torch.full((C,), -1e-3, device=DEV)
    u = _d(z[:, :C])
    half = torch.full((T, C), 0.5, dtype=P.DTYPE)
    want = P.gated_recurrence(u, half, half, torch.full((C,), math.log(math.expm1(1e-3 / 8.0)), dtype=P.DTYPE)) * P.gelu_tanh(_d(z[:, C:]))
    without = P.gated_recurrence(u[1:], half[1:], half[1:], torch.full((C,), math.log(math.expm1(1e-3 / 8.0)), dtype=P.DTYPE))
    assert float((want[1:] / P.gelu_tanh(_d(z[1:, C:])) - without)[-1].abs().max()) > 0.3
    for fused in ([False] if dtype == "float32" else [False, True]):
        for cuts in ([0, T], [0, 1, 3, 130, 257, T], [0, 350] + list(range(351, T + 1))):
            pool = torch.full((2, J * C), float("nan"), device=DEV)
            got = torch.zeros(T, C, dtype=P.DTYPE)
            for first, last in zip(cuts[:-1], cuts[1:]):
                n = last - first
                zs, out = z[first:last].to(DEV), torch.zeros(n, C, dtype=TDT[dtype], device=DEV)
                meta = (_i32([1]), _i32([0, n]), _i32(list(range(first, last))), 1, n)
                if fused and n > 1:
                    assert kernels.diagonal_state_fused(zs, C, conv.t().contiguous(), one, kernels.pack_diagonal_gates(zeros, zeros), S, one, one,
                                                        decay, pool, *meta, out,
                                                        scratch=torch.zeros(kernels.diagonal_fused_scratch_floats(n, C), device=DEV))
                else:
                    uu = torch.zeros(n, C, dtype=TDT[dtype], device=DEV)
                    kernels.short_conv(zs, 0, conv, one, pool[:, C:], meta[0], meta[1], _i32([0] * n), meta[2], 1, uu, 0, n, single=n == 1)
                    kernels.diagonal_state(uu, torch.zeros(n, 2 * C, dtype=TDT[dtype], device=DEV), one, one, decay, S, pool[:, :C], *meta,
                                           out, y=zs[:, C:], scratch=None if n == 1 else
                                           torch.zeros(kernels.diagonal_scratch_floats(n, 1, C), device=DEV))
                got[first:last] = out.cpu().to(P.DTYPE)
            helpers.assert_close(got, want, dtype, f"{len(cuts) - 1} portions, fused {fused}")


@pytest.mark.parametrize("taps", [1, 2, 4, 9])
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_short_convolution_of_single_tokens_keeps_its_inputs(dtype, taps):
    """One token a request and step: outputs and kept inputs are those of the two-kernel form, from NaN slots on, with a
    request of the padding between."""
    g = torch.Generator().manual_seed(taps)
    n, C, T = 5, 70, 12
    u = _rnd(g, T, n, C + 9, dtype=dtype)
    w, b = _rnd(g, C, taps).to(DEV), _rnd(g, C).to(DEV)
    pools = [torch.full((n + 1, max(taps - 1, 1) * C), float("nan"), device=DEV) for _ in range(2)]
    slots, cu = _i32([3, 0, -1, 5, 1]), _i32(list(range(n + 1)))
    live = [0, 1, 3, 4]
    for t in range(T):
        outs = []
        for single, pool in zip((False, True), pools):
            out = torch.full((n, C), 9.0, dtype=TDT[dtype], device=DEV)
            kernels.short_conv(u[t].to(DEV), 9, w, b, pool if taps > 1 else None, slots, cu, _i32(list(range(n))), _i32([t] * n), n, out, 0, n,
                               activation="silu" if taps == 2 else None, single=single)
            outs.append(out[live])
        assert torch.equal(*outs)
        if taps > 1 and t >= taps:
            assert torch.equal(pools[0][[0, 1, 3, 5]], pools[1][[0, 1, 3, 5]])
    assert torch.isnan(pools[1][[2, 4]]).all()
    for i in live:
        want = P.short_conv(_d(u[:, i, 9:]), _d(w.cpu()), _d(b.cpu()))[-1]
        if taps == 2:
            want = want * P.sigmoid(want)
        helpers.assert_close(outs[1][live.index(i)], want, dtype, f"request {i}")


# ---------------------------------------------------------------- slopes, cap, window and sink in the attention kernels
def _paged(k, v, page, perm, dtype):
    T, G, D = k.shape
    kp, vp = (torch.full((len(perm), G, page, D), float("nan"), dtype=TDT[dtype]) for _ in range(2))
    for j in range(T):
        kp[perm[j // page], :, j % page], vp[perm[j // page], :, j % page] = k[j], v[j]
    return kp.to(DEV), vp.to(DEV)


def _every_attention_kernel(q, k, v, want, dtype, scale, first, page, what, **mask):
    """The queries from `first` on as one portion on top of cached tokens, and the last one as a single token."""
    T, H, D = q.shape
    g = torch.Generator().manual_seed(T)
    pages = -(-T // page)
    perm = torch.randperm(pages, generator=g)
    kp, vp = _paged(k, v, page, perm, dtype)
    bt = perm.to(torch.int32).view(1, pages).to(DEV)
    n = T - first
    qd, ref = q[first:].reshape(n, H * D).to(DEV), want[first:].reshape(n, H * D)
    out = torch.zeros(n, H * D, dtype=TDT[dtype], device=DEV)
    kernels.paged_attention_generic(qd, out, kp, vp, bt, _i32([0, n]), _i32([T]), _i32([0] * n), n, 1, H, scale, **mask)
    helpers.assert_close(out, ref, dtype, f"general kernel, {what}")
    one = torch.zeros(1, H * D, dtype=TDT[dtype], device=DEV)
    kernels.paged_attention_generic(qd[n - 1:], one, kp, vp, bt, _i32([0, 1]), _i32([T]), _i32([0]), 1, 1, H, scale, **mask)
    helpers.assert_close(one, ref[n - 1:], dtype, f"general kernel, one query, {what}")
    if dtype != "bfloat16" or D not in (32, 64, 96, 128):
        return
    out.zero_()
    assert kernels.prefill_attention_bf16(qd, out, kp, vp, bt, _i32([0, n]), _i32([T]), 1, n, H, scale, **mask)
    helpers.assert_close(out, ref, dtype, f"tile kernel, {what}")
    for fast in (True, False):
        out.zero_()
        assert kernels.paged_attention_split_bf16(qd, out, kp, vp, bt, _i32([0, n]), _i32([T]), _i32([0] * n), n, 1, H, scale,
                                                  fast=fast, **mask)
        helpers.assert_close(out, ref, dtype, f"split kernel, {what}")
    if D != 96:
        one.zero_()
        assert kernels.paged_attention_decode_bf16(qd[n - 1:], one, kp, vp, bt, _i32([T - 1]), _i32([0]), 1, H, scale,
                                                   identity=True, **mask)
        helpers.assert_close(one, ref[n - 1:], dtype, f"decode kernel, {what}")


KERNEL_DIMS = [("float32", 32), ("bfloat16", 32), ("bfloat16", 64), ("bfloat16", 96), ("bfloat16", 128), ("float32", 20)]


@pytest.mark.parametrize("dtype,D", KERNEL_DIMS)
@pytest.mark.parametrize("window,T,cap", [(1, 40, 6.0), (7, 77, 0.0), (16, 209, 30.0), (17, 205, 6.0), (70, 208, 0.0), (130, 262, 12.0),
                                          (200, 200, 6.0), (300, 210, 30.0), (0, 330, 8.0), (0, 190, 0.0)])
def test_slopes_cap_window_and_sink(dtype, D, window, T, cap):
    """The last query is made to look like one key, scaled so that it takes most of the weight if it is seen: the
    window's first key, then the one before it, then a near one; steep and flat slopes side by side, a sink of score 0 and
    others far above and below."""
    H, G, scale = 4, 2, D ** -0.5
    begin = max(0, T - window) if window else 0
    slope = torch.tensor([0.7, 0.02, 0.001, 0.0])
    for far in (begin, begin - 1, T - 2):
        if far < 0:
            continue
        g = torch.Generator().manual_seed(7 + D + window)
        q, k, v = _rnd(g, T, H, D, dtype=dtype), _rnd(g, T, G, D, dtype=dtype), _rnd(g, T, G, D, dtype=dtype)
        k[far] *= 2.0
        q[-1] = (k[far].float().repeat_interleave(H // G, dim=0) * 3.0).to(TDT[dtype])
        for sink in (0.0, 5.0, None):
            want = P.window_attention(_d(q), _d(k), _d(v), scale, cap, _d(slope), window, sink)
            if far < begin and sink == 0.0:
                seen = P.window_attention(_d(q), _d(k), _d(v), scale, cap, _d(slope), window + 1, sink)
                assert float((want[-1] - seen[-1]).abs().max()) > 0.3      # one position more and the key would take over
            sinks = None if sink is None else torch.full((H,), sink, device=DEV)
            _every_attention_kernel(q, k, v, want, dtype, scale, min(100, T // 2), 16, f"window {window}, cap {cap}, key {far} of {T}, sink {sink}",
                                    window=window, softcap=cap, slopes=slope.to(DEV), sinks=sinks)


@pytest.mark.parametrize("dtype,D", [("float32", 32), ("bfloat16", 64), ("bfloat16", 128)])
def test_slopes_over_many_keys(dtype, D):
    """Hundreds of keys, a sharp one far away that a flat slope lets through and a steep one does not."""
    T, H, G, scale, slope = 700, 8, 1, D ** -0.5, P.slopes(8)
    g = torch.Generator().manual_seed(D)
    q, k, v = _rnd(g, T, H, D, dtype=dtype, scale=0.5), _rnd(g, T, G, D, dtype=dtype, scale=0.5), _rnd(g, T, G, D, dtype=dtype)
    k[20] *= 5.0
    q[600:] = (k[20].float() * 2.0).to(TDT[dtype])
    want = P.window_attention(_d(q), _d(k), _d(v), scale, 25.0, slope, 0)
    flat, steep = (float((want[-1, a] - _d(v)[20, 0]).abs().max()) for a in (7, 0))
    assert flat < 0.5 < steep
    for first in (0, 500, T - 2):
        _every_attention_kernel(q, k, v, want, dtype, scale, first, 16, f"from {first}", softcap=25.0, slopes=slope.float().to(DEV),
                                sinks=torch.zeros(H, device=DEV))


def test_slopes_in_steps_of_several_requests():
    """Portions of different lengths on top of different contexts in one launch of the tile kernel, and single tokens
    of different lengths in one launch of the decode kernel."""
    dtype, D, H, G, page, window, scale, cap = "bfloat16", 64, 3, 1, 16, 48, 0.125, 9.0
    g = torch.Generator().manual_seed(3)
    lens, new = [70, 33, 200, 1, 97], [70, 2, 130, 1, 1]
    slope = torch.tensor([0.3, 0.05, 0.004])
    n_pages = sum(-(-n // page) for n in lens)
    perm = torch.randperm(n_pages, generator=g)
    kp, vp = (torch.full((n_pages, G, page, D), float("nan"), dtype=torch.bfloat16) for _ in range(2))
    bt = torch.full((len(lens), 16), -1, dtype=torch.int32)
    qs, wants, at = [], [], 0
    for r, T in enumerate(lens):
        q, k, v = _rnd(g, T, H, D, dtype=dtype), _rnd(g, T, G, D, dtype=dtype), _rnd(g, T, G, D, dtype=dtype)
        pages = perm[at:at + -(-T // page)]
        at += len(pages)
        bt[r, :len(pages)] = pages.to(torch.int32)
        for j in range(T):
            kp[pages[j // page], :, j % page], vp[pages[j // page], :, j % page] = k[j], v[j]
        qs.append(q)
        wants.append(P.window_attention(_d(q), _d(k), _d(v), scale, cap, _d(slope), window))
    kp, vp, bt = kp.to(DEV), vp.to(DEV), bt.to(DEV)
    mask = dict(window=window, softcap=cap, slopes=slope.to(DEV), sinks=torch.zeros(H, device=DEV))
    rows = torch.cat([q[T - n:] for q, T, n in zip(qs, lens, new)]).reshape(-1, H * D).to(DEV)
    want = torch.cat([w[T - n:] for w, T, n in zip(wants, lens, new)]).reshape(-1, H * D)
    cu = np.concatenate([[0], np.cumsum(new)])
    out = torch.zeros_like(rows)
    assert kernels.prefill_attention_bf16(rows, out, kp, vp, bt, _i32(cu.tolist()), _i32(lens), len(lens), max(new), H, scale, **mask)
    helpers.assert_close(out, want, dtype, "portions of several requests")
    rows = torch.stack([q[-1] for q in qs]).reshape(-1, H * D).to(DEV)
    want = torch.stack([w[-1] for w in wants]).reshape(-1, H * D)
    for ident in (True, False):
        out = torch.zeros_like(rows)
        assert kernels.paged_attention_decode_bf16(rows, out, kp, vp, bt, _i32([n - 1 for n in lens]), _i32(list(range(5))), 5, H, scale,
                                                   identity=ident, **mask)
        helpers.assert_close(out, want, dtype, "single tokens of several requests")


# ---------------------------------------------------------------- what happens to queries, keys and latents in front of attention
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("n,H,G,D,stride,rot", [(3, 4, 2, 24, 32, 0), (70, 6, 1, 64, 64, 16), (5, 2, 2, 20, 24, 20), (90, 1, 1, 128, 128, 128)])
def test_query_temperature_interleaved_rotation_and_values_from_keys(dtype, n, H, G, D, stride, rot):
    g = torch.Generator().manual_seed(n)
    every, coef, eps, page, base = 7, 0.6, 1e-5, 4, 100.0
    z = torch.zeros(n, (H + G) * stride + 5, dtype=TDT[dtype])
    heads = z[:, :(H + G) * stride].view(n, H + G, stride)
    heads[:, :, :D] = _rnd(g, n, H + G, D, dtype=dtype, scale=2.0)
    qn, kn = 1.0 + 0.2 * _rnd(g, D), 1.0 + 0.2 * _rnd(g, D)
    rows = _d(heads[:, :, :D])
    k_raw = rows[:, H:].clone()
    normed = torch.cat([P.rms_norm(rows[:, :H], _d(qn), eps), P.rms_norm(rows[:, H:], _d(kn), eps)], dim=1)
    if rot:
        normed = torch.cat([P.rotate_pairs(normed[..., :rot], base), normed[..., rot:]], dim=-1)
    q = normed[:, :H] * P.query_temperature(n, coef, every)[:, None, None]
    slots = torch.randperm(-(-n // page) * page, generator=g)[:n].to(torch.int32)
    kp, vp = (torch.full((-(-n // page), G, page, stride), 9.0, dtype=TDT[dtype], device=DEV) for _ in range(2))
    freq = torch.tensor([base ** (-2.0 * i / rot) for i in range(rot // 2)], dtype=torch.float64).float().to(DEV) if rot else None
    zd = z.to(DEV)
    kernels.qk_prepare(zd, 0, H * stride, (H + G) * stride, H, G, D, D, stride, n, positions=_i32(list(range(n))), freq=freq, norm_eps=eps,
                       k_pool=kp, v_pool=vp, slot_mapping=slots.to(DEV), norm="head", q_norm_weight=qn.to(DEV), k_norm_weight=kn.to(DEV),
                       values_from_keys=True, interleaved=True, query_temperature=(coef, every))
    helpers.assert_close(zd[:, :H * stride].view(n, H, stride)[:, :, :D], q, dtype, "queries")
    at = slots.long()
    for pool, ref, what in ((kp, normed[:, H:], "keys"), (vp, k_raw, "values")):
        got = pool.permute(0, 2, 1, 3).reshape(-1, G, stride)[at.to(DEV)]
        helpers.assert_close(got[:, :, :D], ref, dtype, what)
        assert (got[:, :, D:] == 0).all()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("n,H,D,R2,R,Q,row", [(5, 3, 12, 8, 24, 40, 32), (33, 1, 20, 6, 100, 16, 128), (2, 4, 4, 64, 512, 300, 576)])
def test_latents_of_keys_and_of_queries_with_interleaved_pairs(dtype, n, H, D, R2, R, Q, row):
    g = torch.Generator().manual_seed(n)
    eps, base, page = 1e-5, 50.0, 4
    z = _rnd(g, n, Q + R + R2 + 3, dtype=dtype)
    q = _rnd(g, n, H * (D + R2) + 2, dtype=dtype)
    gain, cq_gain = 1.0 + 0.2 * _rnd(g, R), 1.0 + 0.2 * _rnd(g, Q)
    freq = torch.tensor([base ** (-2.0 * i / R2) for i in range(R2 // 2)], dtype=torch.float64).float().to(DEV)
    slots = torch.randperm(-(-n // page) * page, generator=g)[:n].to(torch.int32)
    slots[n - 1] = -1                        # a token of the padding
    pool = torch.full((-(-n // page), 1, page, row), 9.0, dtype=TDT[dtype], device=DEV)
    cq = torch.full((n + 1, Q), 9.0, dtype=TDT[dtype], device=DEV)
    zd, pos = z.to(DEV), _i32(list(range(n)))
    kernels.latent_prepare(zd, 0, 0, D, R2, pos, freq, n, c_off=Q, rank=R, gain=gain.to(DEV), eps=eps, pool=pool, slot_mapping=slots.to(DEV),
                           interleaved=True, cq_gain=cq_gain.to(DEV), cq_out=cq)
    assert torch.equal(zd.cpu(), z) and (cq[n] == 9.0).all()
    helpers.assert_close(cq[:n], P.rms_norm(_d(z[:, :Q]), _d(cq_gain), eps), dtype, "the queries' latent")
    want = torch.cat([P.rms_norm(_d(z[:, Q:Q + R]), _d(gain), eps), P.rotate_pairs(_d(z[:, Q + R:Q + R + R2]), base)], dim=1)
    got = pool.view(-1, row)[slots[:n - 1].long().to(DEV)]
    helpers.assert_close(got[:, :R + R2], want[:n - 1], dtype, "cached rows")
    assert (got[:, R + R2:] == 0).all()
    untouched = [s for s in range(pool.shape[0] * page) if s not in slots.tolist()]
    assert (pool.view(-1, row)[untouched] == 9.0).all()
    qd = q.to(DEV)
    kernels.latent_prepare(qd, 2, H, D, R2, pos, freq, n, interleaved=True)
    heads = _d(q[:, 2:]).view(n, H, D + R2)
    want = torch.cat([heads[..., :D], P.rotate_pairs(heads[..., D:], base)], dim=-1)
    helpers.assert_close(qd[:, 2:], want.reshape(n, -1), dtype, "queries")


@pytest.mark.parametrize("n,H,D,R2,row", [(1, 2, 16, 8, 64), (8, 16, 96, 32, 128), (70, 3, 8, 16, 32), (300, 4, 40, 64, 128)])
def test_folding_product_turns_the_queries_rotated_part(n, H, D, R2, row):
    g = torch.Generator().manual_seed(n)
    base = 30.0
    q, w = _rnd(g, n, H * (D + R2) + 8, dtype="bfloat16"), _rnd(g, H, row, D + R2, dtype="bfloat16", scale=(D + R2) ** -0.5)
    freq = torch.tensor([base ** (-2.0 * i / R2) for i in range(R2 // 2)], dtype=torch.float64).float().to(DEV)
    turns = torch.full((n, R2), 9.0, device=DEV)
    kernels.latent_prepare(q.to(DEV), 0, 0, D, R2, _i32(list(range(n))), freq, n, turns=turns, interleaved=True)
    a = torch.arange(n, dtype=P.DTYPE)[:, None] * _d(freq.cpu())
    helpers.assert_close(turns, torch.cat([torch.cos(a), torch.sin(a)], dim=1), "float32", "cosines and sines")
    out = torch.full((n, H * row), 9.0, dtype=torch.bfloat16, device=DEV)
    assert kernels.heads_linear(q.to(DEV), w.to(DEV), out, n, fast=True, turns=turns)
    heads = _d(q[:, :H * (D + R2)]).view(n, H, D + R2)
    heads = torch.cat([heads[..., :D], P.rotate_pairs(heads[..., D:], base)], dim=-1)
    want = torch.einsum("nhi,hoi->nho", heads, _d(w)).reshape(n, H * row)
    helpers.assert_close(out, want, "bfloat16", "folded queries")
    # parts that are not eight channels at a time are left to others
    odd = torch.zeros(n, 6, device=DEV)
    assert not kernels.heads_linear(q.to(DEV), w[:, :, :D + R2].contiguous().to(DEV), out, n, fast=True, turns=odd)
    assert not kernels.heads_linear(q.float().to(DEV), w.float().to(DEV), out.float(), n, turns=turns)


# ---------------------------------------------------------------- the router, the unit, the norm behind a sublayer
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("n,width,experts,top,groups", [(9, 40, 6, 2, (3, 2)), (70, 264, 12, 3, (4, 1)), (5, 2048, 8, 2, (8, 5)), (4, 24, 3, 3, (1, 1)),
                                                        (33, 136, 64, 4, (8, 4)), (3, 100, 130, 2, (65, 3)), (6, 64, 256, 8, (8, 2)), (2, 64, 1, 1, (1, 1))])
def test_router_with_softmax_scores_and_groups_by_their_best(dtype, n, width, experts, top, groups):
    g = torch.Generator().manual_seed(n + experts)
    h = _rnd(g, n + 1, width + 8, dtype=dtype)
    w = _rnd(g, experts, width, dtype=dtype, scale=width ** -0.5 * 3.0)
    scores = torch.softmax(_d(h[:n, :width]) @ _d(w).T, dim=-1)
    P.ROUTER_GAPS = []
    try:
        want = P.grouped_choice(scores, top, *groups)
        firm = P.ROUTER_GAPS[0] > 1e-4
    finally:
        P.ROUTER_GAPS = None
    assert int(firm.sum()) >= n - 1
    raw = torch.gather(scores, 1, want)
    chosen = torch.full((n + 1, top), -7, dtype=torch.int32, device=DEV)
    weight = torch.full((n + 1, top), -7.0, device=DEV)
    for normalise in (True, False):
        kernels.router_topk(h.to(DEV), w.to(DEV), n, top, chosen, weight, score="softmax", groups=groups, normalise=normalise, group_best=1)
        assert (chosen[n] == -7).all() and (weight[n] == -7.0).all()
        assert torch.equal(chosen[:n].cpu().long()[firm], want[firm])
        ref = raw / (raw.sum(dim=1, keepdim=True) + 1e-20) if normalise else raw
        helpers.assert_close(weight[:n].cpu()[firm], ref[firm], "float32", f"weights, normalise {normalise}")


@pytest.mark.parametrize("dtype", ["bfloat16"])
@pytest.mark.parametrize("n,width,experts,top,tile", [(1, 64, 4, 2, 16), (8, 2048, 8, 2, 16), (16, 264, 64, 5, 16), (5, 40, 12, 3, 64), (3, 24, 1, 1, 16)])
def test_router_that_sorts_its_pairs_in_the_same_launch(dtype, n, width, experts, top, tile):
    """Choice and weights are the separate kernels' (with softmax, sigmoid scores with a correction, a shared expert's
    number), every pair has a slot in a tile of its expert, and a token of the padding has none."""
    g = torch.Generator().manual_seed(n + experts)
    h, w = _rnd(g, n, width, dtype=dtype).to(DEV), _rnd(g, experts, width, dtype=dtype, scale=2.0 * width ** -0.5).to(DEV)
    extra, correction = _rnd(g, 1, width, dtype=dtype).to(DEV), _rnd(g, experts).to(DEV)
    q_req = _i32([-1 if i == n // 2 and n > 1 else i for i in range(n)])
    live = [i for i in range(n) if not (i == n // 2 and n > 1)]
    slots = kernels.expert_slots(n, top, experts, tile)
    for rule in (dict(score="softmax", normalise=True, group_best=1, groups=(experts, experts)),
                 dict(score="sigmoid", correction=correction, normalise=True, scale=1.5),
                 dict(score="softmax", group_best=1, groups=(2, 1)) if experts % 2 == 0 and top <= experts // 2 else dict(score="logit")):
        outs = []
        for sort in (False, True):
            chosen, weight = torch.full((n, top), -7, dtype=torch.int32, device=DEV), torch.full((n, top), -7.0, device=DEV)
            gate = torch.full((n,), -7.0, device=DEV)
            st, sp, te = (torch.full((k,), -9, dtype=torch.int32, device=DEV) for k in (slots, slots, slots // tile))
            assert kernels.router_topk(h, w, n, top, chosen, weight, q_req=q_req, extra=extra, extra_out=gate,
                                       slots=(st, sp, te, slots, tile) if sort else None, **rule)
            outs.append((chosen, weight, gate))
        assert torch.equal(outs[0][0], outs[1][0])
        for a, b in zip(outs[0][1:], outs[1][1:]):
            helpers.assert_close(a, b, "float32", str(rule))
        st, sp, te = st.tolist(), sp.tolist(), te.tolist()
        used = [s for s in range(slots) if st[s] >= 0]
        assert sorted(sp[s] for s in used) == [i * top + c for i in live for c in range(top)]
        for s in used:
            assert st[s] == sp[s] // top and te[s // tile] == int(outs[1][0][st[s], sp[s] % top])
        assert all(te[t] == -1 for t in range(slots // tile) if all(st[s] < 0 for s in range(t * tile, (t + 1) * tile)))
    assert not kernels.router_topk(h.float(), w.float(), n, top, chosen, weight, slots=(*(torch.zeros(k, dtype=torch.int32, device=DEV) for k in
                                                                                         (slots, slots, slots // tile)), slots, tile))
    assert not kernels.router_topk(h.repeat(17, 1), w, 17, top, torch.zeros(17, top, dtype=torch.int32, device=DEV), torch.zeros(17, top, device=DEV),
                                   slots=(torch.zeros(17 * top * tile, dtype=torch.int32, device=DEV),) * 2
                                   + (torch.zeros(17 * top, dtype=torch.int32, device=DEV), 17 * top * tile, tile))


def test_a_group_by_its_best_and_by_its_two_best_differ():
    """Group 0 has the best expert and nothing else, groups 1 and 2 two good ones each."""
    logits = torch.tensor([[3.0, -9.0, 2.5, 2.4, 2.45, 2.3]])
    h, w = torch.eye(6)[:1].to(DEV), torch.zeros(6, 6)
    w[:, 0] = logits[0]
    got = {}
    for best in (1, 2):
        chosen, weight = torch.zeros(1, 2, dtype=torch.int32, device=DEV), torch.zeros(1, 2, device=DEV)
        kernels.router_topk(h, w.to(DEV), 1, 2, chosen, weight, score="softmax", groups=(3, 2), group_best=best)
        got[best] = sorted(chosen[0].tolist())
    assert got == {1: [0, 2], 2: [2, 4]}
    chosen, weight = torch.zeros(1, 2, dtype=torch.int32, device=DEV), torch.zeros(1, 2, device=DEV)
    # by the two best of every group (of logits, which may be negative) the first group is out
    kernels.router_topk(h, w.to(DEV), 1, 2, chosen, weight, score="logit", groups=(3, 2), group_best=2)
    assert sorted(chosen[0].tolist()) == [2, 4]


def test_softmax_scores_of_very_different_logits():
    logits = torch.tensor([[200.0, 90.0, -300.0, 199.0, 0.0]])
    h, w = torch.ones(1, 1).to(DEV), logits.t().contiguous().to(DEV)
    chosen, weight = torch.zeros(1, 3, dtype=torch.int32, device=DEV), torch.zeros(1, 3, device=DEV)
    kernels.router_topk(h, w, 1, 3, chosen, weight, score="softmax", normalise=True)
    assert chosen[0].tolist() == [0, 3, 1]
    helpers.assert_close(weight, torch.softmax(_d(logits), dim=-1)[:, [0, 3, 1]], "float32", "scores")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("n,hidden,limit,sharpness", [(5, 40, 1.5, 1.702), (3, 37, 0.4, 1.702), (70, 128, 7.0, 1.0)])
def test_clamped_swish_unit(dtype, n, hidden, limit, sharpness):
    g = torch.Generator().manual_seed(hidden)
    z = _rnd(g, n + 1, 2 * hidden + 8, dtype=dtype, scale=2.0 * limit)
    act = torch.full((n + 1, hidden), 9.0, dtype=TDT[dtype], device=DEV)
    gate, up = torch.clamp(_d(z[:n, :hidden]), max=limit), torch.clamp(_d(z[:n, hidden:2 * hidden]), -limit, limit)
    want = gate * P.sigmoid(sharpness * gate) * (up + 1.0)
    for fast in (False, True):
        kernels.gated_unit(z.to(DEV), act, n, hidden, fast=fast, activation="clamped_swish", limit=limit, sharpness=sharpness)
        assert (act[n] == 9.0).all()
        helpers.assert_close(act[:n], want, dtype, f"unit, fast {fast}")


UNITS = {"silu": lambda g, u: g * P.sigmoid(g) * u, "relu": lambda g, u: torch.clamp(g, min=0.0) * u,
         "gelu_tanh": lambda g, u: P.gelu_tanh(g) * u, "clamped_swish": lambda g, u: P.clamped_swish_unit(g, u, 0.9)}


@pytest.mark.parametrize("activation", sorted(UNITS))
@pytest.mark.parametrize("n,width,hidden", [(1, 64, 48), (5, 40, 37), (16, 2048, 1360), (7, 520, 16), (3, 1000, 100)])
def test_gated_products_of_few_rows_with_their_unit(activation, n, width, hidden):
    """One matrix pair for all rows, and pairs of four experts in tiles of 16 slots, gathered and in order; inner sizes with
    and without a rest of less than 32; and the product without a unit, float32 out at places of its own."""
    g = torch.Generator().manual_seed(n + width)
    extra = {"limit": 0.9, "sharpness": 1.702} if activation == "clamped_swish" else {}
    h = _rnd(g, n + 1, width + 8, dtype="bfloat16")
    w = _rnd(g, 4, 2 * hidden, width, dtype="bfloat16", scale=width ** -0.5)
    rows = _d(h[:n, :width])
    want = torch.stack([UNITS[activation](rows @ _d(w[e, :hidden]).T, rows @ _d(w[e, hidden:]).T) for e in range(4)])
    act = torch.full((n + 1, hidden), 9.0, dtype=torch.bfloat16, device=DEV)
    assert kernels.gated_few_rows(h.to(DEV), w[2].to(DEV), act, n, hidden, activation=activation, **extra)
    assert (act[n] == 9.0).all()
    helpers.assert_close(act[:n], want[2], "bfloat16", "one matrix pair")
    table = torch.stack([torch.randperm(4, generator=g)[:2] for _ in range(n)]).to(torch.int32)
    slots = kernels.expert_slots(n, 2, 4, 16)
    st, sp, te = (torch.zeros(k, dtype=torch.int32, device=DEV) for k in (slots, slots, slots // 16))
    kernels.expert_route(None, None, table.to(DEV), n, 4, st, sp, te, 16)
    used = (st >= 0).nonzero().flatten().tolist()
    ref = torch.stack([want[table[st[s], sp[s] % 2], st[s]] for s in used])
    ordered = torch.zeros(slots, width, dtype=torch.bfloat16, device=DEV)
    ordered[used] = h[st[used].cpu().long(), :width].to(DEV)
    for a, a_rows in ((h.to(DEV), st), (ordered, None)):
        act = torch.full((slots, hidden), 9.0, dtype=torch.bfloat16, device=DEV)
        assert kernels.gated_few_rows(a, w.to(DEV), act, 0, hidden, a_rows=a_rows, tile_expert=te, slot_token=st, n_slots=slots,
                                      activation=activation, **extra)
        helpers.assert_close(act[used], ref, "bfloat16", "experts")
        assert (act[[s for s in range(slots) if s not in used]] == 9.0).all()
    # tiles of 16 without a unit
    down = _rnd(g, 4, 24, width, dtype="bfloat16", scale=width ** -0.5)
    out = torch.full((2 * n, 24), 9.0, device=DEV)
    kernels.grouped_linear(h.to(DEV)[:, :width], st, down.to(DEV), te, st, out, sp, slots, 16, True)
    ref = torch.stack([rows[t] @ _d(down[table[t, c]]).T for t in range(n) for c in range(2)])
    helpers.assert_close(out, ref, "bfloat16", "without a unit")


def test_gated_products_of_more_rows_are_left_to_other_kernels():
    h, w = torch.zeros(17, 64, dtype=torch.bfloat16, device=DEV), torch.zeros(32, 64, dtype=torch.bfloat16, device=DEV)
    act = torch.zeros(17, 16, dtype=torch.bfloat16, device=DEV)
    assert not kernels.gated_few_rows(h, w, act, 17, 16)
    assert not kernels.gated_few_rows(h.float(), w.float(), act.float(), 4, 16)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("width", [40, 1024, 3000, 5000])
def test_norm_behind_a_sublayer_hands_the_residual_on(dtype, width):
    g = torch.Generator().manual_seed(width)
    n, eps = 5, 1e-5
    x, y, gain = _rnd(g, n + 1, width), _rnd(g, n + 1, width, scale=3.0), 1.0 + 0.1 * _rnd(g, width)
    xd, yd = x.to(DEV), y.to(DEV)
    h = torch.full((n + 1, width), 9.0, dtype=TDT[dtype], device=DEV)
    kernels.cast_rows(xd, h, n, width)
    assert torch.equal(h[:n].cpu(), x[:n].to(TDT[dtype])) and (h[n] == 9.0).all()
    kernels.rms_post_norm([(yd, None)], xd, gain.to(DEV), n, eps, 0.0, 1.0, h=h)
    want = _d(x[:n]) + P.rms_norm(_d(y[:n]), _d(gain), eps)
    helpers.assert_close(xd[:n], want, "float32", "residual")
    assert torch.equal(h[:n], xd[:n].to(TDT[dtype])) and (h[n] == 9.0).all()
    assert (yd[:n] == 0).all() and torch.equal(yd[n].cpu(), y[n]) and torch.equal(xd[n].cpu(), x[n])


# ---------------------------------------------------------------- the model through the step function
LENGTHS = {"A": [5, 70, 23, 41, 2, 64, 37], "B": [1, 9, 33, 17, 140], "C": [40, 3, 64, 21], "D": [75, 12, 30, 6, 49],
           "E": [33, 4, 70, 18, 2, 131], "F": [130, 1, 66, 40, 9]}
_folders, _plain, _twin = {}, {}, {}


def _folder(tmp_path_factory, name):
    if name not in _folders:
        _folders[name] = cases.write_model(str(tmp_path_factory.mktemp("telapel") / name), name)
    return _folders[name]


FIRM_GAP = 0.25     # between router logits: a choice decided by less is no test of reduced precision


def _router_gaps(cfg, w, ids):
    """Per position: by how much the least decided router's choice is decided in the plain implementation."""
    P.ROUTER_GAPS = []
    try:
        P.forward(cfg, w, ids)
        gaps = torch.stack(P.ROUTER_GAPS).min(dim=0).values if P.ROUTER_GAPS else torch.full((len(ids),), math.inf)
    finally:
        P.ROUTER_GAPS = None
    return gaps.numpy()


def _firm_ids(cfg, w, rng, vocab, n):
    """n random tokens, each drawn again (up to 50 times) until every router's choice at its position is decided by
    FIRM_GAP: rounding to bfloat16 then chooses the same experts, and the logits can be compared.  (A position's
    routing depends on the tokens up to it only.)"""
    ids = []
    while len(ids) < n:
        for _ in range(50):
            tok = int(rng.integers(0, vocab))
            if _router_gaps(cfg, w, ids + [tok])[-1] >= FIRM_GAP:
                break
        ids.append(tok)
    return ids


def _firm_prefix(cfg, w, ids):
    """The number of positions before the first whose routing is a close call."""
    close = np.nonzero(_router_gaps(cfg, w, ids) < FIRM_GAP)[0]
    return int(close[0]) if len(close) else len(ids)


_requests_made = {}


def _requests(folder, name):
    if name not in _requests_made:
        cfg, w = P.read_model_folder(folder)
        rng = np.random.default_rng(len(name) + ord(name[0]))
        _requests_made[name] = {f"r{i}": _firm_ids(cfg, w, rng, cases.RAW[name]["vocab"], n)
                                for i, n in enumerate(LENGTHS[name])}
    return _requests_made[name]


def _plain_logits(folder, name):
    if name not in _plain:
        cfg, w = P.read_model_folder(folder)
        _plain[name] = {rid: P.forward(cfg, w, ids).numpy() for rid, ids in _requests(folder, name).items()}
    return _plain[name]


def _row_errors(got, want):
    """Per position: root mean square over the vocabulary of the difference, its mean taken off."""
    d = np.asarray(got, dtype=np.float64) - np.asarray(want, dtype=np.float64)
    d = d - d.mean(axis=1, keepdims=True)
    return np.sqrt((d * d).mean(axis=1))


def _rounded_twin(cfg, w, ids):
    """The plain implementation with every matrix product rounded to bfloat16: what rounding alone does."""
    P.ROUNDING = torch.bfloat16
    try:
        return P.forward(cfg, w, ids).numpy()
    finally:
        P.ROUNDING = None


def _assert_within_rounding(folder, key, ids, got, want, what, worst=3.0, upto=None):
    """bfloat16: a position's error may be `worst` times what rounding alone causes at the request's
    worst position, and the request's mean error three times the mean of that (over the first `upto` positions)."""
    assert np.isfinite(got).all(), f"{what}: non-finite logits"
    if key not in _twin:
        cfg, w = P.read_model_folder(folder)
        _twin[key] = _row_errors(_rounded_twin(cfg, w, ids), want)
    noise, err = _twin[key][:upto], _row_errors(got, want)[:upto]
    assert err.max() <= worst * noise.max(), f"{what}: worst position {err.max():.3e} > {worst} * {noise.max():.3e}"
    assert err.mean() <= 3.0 * noise.mean(), f"{what}: mean {err.mean():.3e} > 3 * {noise.mean():.3e}"


def _check(folder, name, dtype, rid, ids, got, want, what, upto=None):
    if dtype == "float32":
        assert np.isfinite(got).all(), what
        err = _row_errors(got, want)
        assert err.max() <= 5e-5 * max(1.0, float(np.abs(want).max())), f"{what}: {err.max():.3e}"
    else:
        _assert_within_rounding(folder, (name, rid, len(ids)), ids, got, want, what, upto=upto)


@pytest.mark.parametrize("page_size", [16, 4])
@pytest.mark.parametrize("way", ["whole", "tail", "portions", "mixed"])
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", sorted(cases.RAW))
def test_every_way_of_cutting_matches_the_plain_implementation(tmp_path_factory, name, dtype, way, page_size):
    folder = _folder(tmp_path_factory, name)
    reqs = _requests(folder, name)
    want = _plain_logits(folder, name)
    plan = helpers.PLANS[way](reqs, np.random.default_rng(5))
    # the pool holds just what the live requests need and starts as NaN, and so do the states; four request slots
    replayer = TraceReplayer(folder, dtype, plan.tight_tokens(page_size), page_size=page_size, max_live=4, poison=True)
    got = plan.assemble(helpers.run_plan_in_process(replayer, plan), {r: len(t) for r, t in reqs.items()},
                        cases.RAW[name]["vocab"])
    for rid in reqs:
        _check(folder, name, dtype, rid, reqs[rid], got[rid], want[rid], f"{name} {dtype} {way} {rid}")
    assert replayer.cache.check() == 0 and not replayer.live
    assert all(replayer.cache.num_free_pages(g) == replayer.num_pages for g in range(len(replayer.cache.groups)))


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["A", "B"])
def test_steps_that_want_no_logits_leave_the_state_right(tmp_path_factory, name, dtype):
    """Token-by-token steps of which only every fourth wants its logits, and mixed steps likewise:
    step shapes come back often enough to be replayed from recorded launches and from graphs, and a
    request's states and kept convolution inputs must have seen every token once."""
    folder = _folder(tmp_path_factory, name)
    reqs = _requests(folder, name)
    want = _plain_logits(folder, name)
    cfg, w = P.read_model_folder(folder)
    noise = {rid: _row_errors(_rounded_twin(cfg, w, ids), want[rid]).max() for rid, ids in reqs.items()}
    for way in ("tail", "mixed"):
        plan = helpers.PLANS[way](reqs, np.random.default_rng(7))
        kept = {}
        for rec in plan.steps:
            rows, keep, at = plan.wanted[rec["step"]], [], 0
            for entry in rec["entries"]:
                n = len(entry["tokens"])
                entry["want"] = [i for i in range(n) if (rec["step"] + i) % 4 == 0]
                keep += [rows[at + i] for i in entry["want"]]
                at += n
            kept[rec["step"]] = keep
        plan.wanted = {s: rows for s, rows in kept.items() if rows}
        replayer = TraceReplayer(folder, dtype, plan.tight_tokens(16), page_size=16, max_live=4, poison=True)
        outputs = helpers.run_plan_in_process(replayer, plan)
        vocab = cases.RAW[name]["vocab"]
        for step, rows in plan.wanted.items():
            out = np.asarray(outputs[step], dtype=np.float64).reshape(len(rows), vocab)
            for (rid, pos), row in zip(rows, out):
                ref = want[rid][pos:pos + 1]
                err = float(_row_errors(row[None], ref)[0])
                bound = 5e-5 * max(1.0, float(np.abs(ref).max())) if dtype == "float32" else 3.0 * noise[rid]
                assert np.isfinite(row).all() and err <= bound, f"{name} {dtype} {way} {rid} position {pos}: {err:.3e}"


@pytest.mark.parametrize("seed", range(8))
def test_random_configurations(tmp_path, seed):
    """Configurations drawn at random (tests/telapel_cases.py: random_raw), five requests of lengths
    1 to 200 each, whole, in portions and mixed, in both dtypes.  bfloat16: a position may be one and
    a half times over three times what rounding alone does, the mean may not; a request is compared up to
    its first position where a router's choice is a close call."""
    rng = np.random.default_rng(5000 + seed)
    raw = cases.random_raw(rng)
    folder = cases.write_raw_model(str(tmp_path / "m"), raw, seed)
    cfg, w = P.read_model_folder(folder)
    lens = [int(x) for x in rng.choice([1, 2, 5, 17, 33, 64, 70, 97, 130, 200], size=5)]
    reqs = {f"r{i}": helpers.random_ids(rng, raw["vocab"], n) for i, n in enumerate(lens)}
    want = {rid: P.forward(cfg, w, ids).numpy() for rid, ids in reqs.items()}
    noise = {rid: _row_errors(_rounded_twin(cfg, w, ids), want[rid]) for rid, ids in reqs.items()}
    firm = {rid: _firm_prefix(cfg, w, ids) for rid, ids in reqs.items()}
    for dtype in ("float32", "bfloat16"):
        for way in ("whole", "portions", "mixed"):
            plan = helpers.PLANS[way](reqs, np.random.default_rng(5))
            replayer = TraceReplayer(folder, dtype, plan.tight_tokens(16), page_size=16, max_live=4, poison=True)
            got = plan.assemble(helpers.run_plan_in_process(replayer, plan), {r: len(t) for r, t in reqs.items()},
                                raw["vocab"])
            for rid in reqs:
                what = f"seed {seed} {dtype} {way} {rid} ({json.dumps(raw)})"
                assert np.isfinite(got[rid]).all(), what
                err = _row_errors(got[rid], want[rid])
                if dtype == "float32":
                    assert err.max() <= 5e-5 * max(1.0, float(np.abs(want[rid]).max())), f"{err.max():.3e}: {what}"
                    continue
                # bfloat16 may choose other experts where a router's choice is a close call, and what follows in
                # that request differs too: the positions before the first such call are compared
                if not firm[rid]:
                    continue
                e, nz = err[:firm[rid]], noise[rid][:firm[rid]]
                assert e.max() <= 4.5 * nz.max() and e.mean() <= 3.0 * nz.mean(), \
                    f"{e.max():.3e} / {nz.max():.3e}, mean {e.mean():.3e} / {nz.mean():.3e}: {what}"


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_long_decoding(tmp_path_factory, dtype):
    """Three tokens of prompt, then 300 tokens one by one through pages of four tokens: states and kept
    convolution inputs are carried over hundreds of steps, the window moves over decoded tokens only, the
    temperature rises, the decode steps come from graphs."""
    folder = _folder(tmp_path_factory, "A")
    cfg, w = P.read_model_folder(folder)
    rng = np.random.default_rng(9)
    ids = _firm_ids(cfg, w, rng, cases.RAW["A"]["vocab"], 40) + helpers.random_ids(rng, cases.RAW["A"]["vocab"], 263)
    want = P.forward(cfg, w, ids).numpy()
    plan = helpers.plan_tail({"a": ids}, tail=300)
    replayer = TraceReplayer(folder, dtype, 304, page_size=4, max_live=4, poison=True)
    got = plan.assemble(helpers.run_plan_in_process(replayer, plan), {"a": len(ids)}, cases.RAW["A"]["vocab"])
    # (bfloat16: up to the first position where a router's choice is a close call, all of it in 32-bit)
    upto = None if dtype == "float32" else _firm_prefix(cfg, w, ids)
    assert np.isfinite(got["a"]).all() and (upto is None or upto >= 8)
    _check(folder, "A", dtype, "long", ids, got["a"], want, "long decoding", upto=upto)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_sharp_attention_at_window_edges_prefill_and_decoding(tmp_path, dtype):
    """Configuration D with the query and key gains of its attention layer scaled up (a sharp softmax under the cap): 100
    tokens whole, in portions, and with the last 70 one by one, so that keys leave the window of 33 among prompt tokens
    and among decoded ones."""
    def edit(tensors):
        for n in ("q", "k"):
            tensors[f"l1.mix.{n}.norm"] *= 2.5
    folder = cases.write_model(str(tmp_path / "sharp"), "D", edit=edit)
    cfg, w = P.read_model_folder(folder)
    ids = _firm_ids(cfg, w, np.random.default_rng(11), cases.RAW["D"]["vocab"], 100)
    want = P.forward(cfg, w, ids).numpy()
    # the window matters: one position less and the logits move
    for size in (32, 34):
        other = json.loads(json.dumps(cfg))
        other["layers"][1]["mixer"]["mask"]["size"] = size
        assert _row_errors(P.forward(other, w, ids).numpy(), want)[40:].max() > 1e-2
    for way, plan in (("whole", helpers.plan_whole({"a": ids})), ("portions", helpers.plan_portions({"a": ids}, None)),
                      ("tail", helpers.plan_tail({"a": ids}, tail=70))):
        replayer = TraceReplayer(folder, dtype, 128, page_size=16, max_live=4, poison=True)
        got = plan.assemble(helpers.run_plan_in_process(replayer, plan), {"a": len(ids)}, cases.RAW["D"]["vocab"])
        _check(folder, "sharp", dtype, "a", ids, got["a"], want, f"sharp {dtype} {way}")


@pytest.mark.parametrize("cut", [62, 63, 64, 65, 66])
def test_portions_of_two_around_a_page_and_a_kernels_chunk(tmp_path_factory, cut):
    """Two portions of two tokens each around position 64 (a page's and a recurrence chunk's border), the rest in one
    piece before and one by one behind, in 32-bit."""
    folder = _folder(tmp_path_factory, "D")
    cfg, w = P.read_model_folder(folder)
    ids = helpers.random_ids(np.random.default_rng(cut), cases.RAW["D"]["vocab"], 76)
    want = P.forward(cfg, w, ids).numpy()
    replayer = TraceReplayer(folder, "float32", 128, page_size=16, max_live=4, poison=True)
    got, at = [], 0
    for step, n in enumerate([cut - 2, 2, 2] + [1] * (76 - cut - 2)):
        rec = {"step": step, "entries": [{"id": "a", "tokens": ids[at:at + n], "want": list(range(n))}],
               "end": ["a"] if at + n == 76 else []}
        got.append(replayer.run_step(rec).cpu().numpy())
        at += n
    _check(folder, "D", "float32", "cut", ids, np.concatenate(got), want, f"cut at {cut}")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_a_windows_passed_pages_are_used_again_within_a_request(tmp_path_factory, dtype):
    """A pool far smaller than the request in the window's group would not do for the latents' group, which keeps every
    key: pages of the window's group go back as the window passes them, and the others stay."""
    folder = _folder(tmp_path_factory, "D")
    cfg, w = P.read_model_folder(folder)
    ids = _firm_ids(cfg, w, np.random.default_rng(21), cases.RAW["D"]["vocab"], 60)
    replayer = TraceReplayer(folder, dtype, 64, page_size=4, max_live=4, poison=True)
    got = []
    for at in range(0, 60, 5):
        rec = {"step": at, "entries": [{"id": "a", "tokens": ids[at:at + 5], "want": list(range(5))}], "end": []}
        got.append(replayer.run_step(rec).cpu().numpy())
    layout = replayer.model.cache_layout
    for g, spec in enumerate(layout.groups):
        held = replayer.cache.held_pages(replayer.live["a"][0], g)
        # positions 28 .. 59 may still be seen by the token at 60: eight pages of four, from position 28 on
        assert held == (8 if spec.window else 15)
    _check(folder, "D", dtype, "pages", ids, np.concatenate(got), P.forward(cfg, w, ids).numpy(), "passed pages")


@pytest.mark.parametrize("name", ["A", "B", "E"])
def test_greedy_generation_through_the_engine(tmp_path_factory, name):
    folder = _folder(tmp_path_factory, name)
    cfg, w = P.read_model_folder(folder)
    vocab = cases.RAW[name]["vocab"]
    rng = np.random.default_rng(2)
    prompts = [_firm_ids(cfg, w, rng, vocab, n) for n in (7, 19, 3, 11, 26)]
    want = [P.greedy(cfg, w, p, 10) for p in prompts]
    # three request slots for five prompts, portions of at most 8 tokens, small pages: requests
    # wait, prompts are cut, slots, pages and states are used again
    engine = LLMEngine.from_folder(folder, EngineConfig(block_size=4, num_blocks=48, max_batch_size=3,
                                                        prefill_chunk=8, dtype="float32"))
    got = engine.generate(prompts, SamplingParams(max_tokens=10, temperature=0.0))
    assert got == want
    engine = LLMEngine.from_folder(folder, EngineConfig(block_size=16, num_blocks=32, max_batch_size=3, dtype="bfloat16"))
    got = engine.generate(prompts, SamplingParams(max_tokens=10, temperature=0.0))
    checked = 0
    for prompt, tokens in zip(prompts, got):
        seq = list(prompt)
        assert len(tokens) == 10
        for tok in tokens:
            if _firm_prefix(cfg, w, seq) < len(seq):
                break       # a router's close call: from here on bfloat16 may have gone another, as valid, way
            logits = P.forward(cfg, w, seq)[-1].numpy()
            margin = 2 * helpers.TOL["bfloat16"] * max(1.0, float(abs(logits).max()))
            assert logits[tok] >= logits.max() - margin
            seq.append(tok)
            checked += 1
    assert checked >= 4


def test_generation_with_evictions_recomputes_the_state(tmp_path_factory):
    """A page pool too small for all running requests: the newest is evicted and later recomputed
    from its prompt and outputs, its states and kept convolution inputs starting over; the tokens are
    those of an engine with room."""
    folder = _folder(tmp_path_factory, "D")
    rng = np.random.default_rng(3)
    prompts = [helpers.random_ids(rng, cases.RAW["D"]["vocab"], n) for n in (9, 14, 5, 12)]
    roomy = LLMEngine.from_folder(folder, EngineConfig(block_size=4, num_blocks=64, max_batch_size=4, dtype="float32"))
    want = roomy.generate(prompts, SamplingParams(max_tokens=24, temperature=0.0))
    tight = LLMEngine.from_folder(folder, EngineConfig(block_size=4, num_blocks=22, max_batch_size=4, dtype="float32"))
    got = tight.generate(prompts, SamplingParams(max_tokens=24, temperature=0.0))
    assert got == want
    assert tight.stats()["num_preemptions"] > 0


def test_the_command_line_and_seeded_sampling(tmp_path_factory):
    """`python -m mini_gpt_inference_amd.generate` on a Telapel folder: the architecture is found by config.json,
    greedy tokens are the plain implementation's; sampling with a seed through the engine gives the same tokens
    whatever the batch a request runs in."""
    folder = _folder(tmp_path_factory, "D")
    cfg, w = P.read_model_folder(folder)
    prompt = [5, 17, 3, 20]
    want = P.greedy(cfg, w, prompt, 6)
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    proc = subprocess.run([sys.executable, "-m", "mini_gpt_inference_amd.generate", "--model", folder,
                           "--prompt-ids", ",".join(map(str, prompt)), "--max-new-tokens", "6", "--temperature", "0",
                           "--dtype", "float32", "--kv-block-size", "4", "--num-kv-blocks", "32"],
                          cwd=root, capture_output=True, text=True, timeout=300)
    assert proc.returncode == 0, proc.stderr[-2000:]
    assert "Telapel" in proc.stdout
    line = next(l for l in proc.stdout.splitlines() if l.startswith("sample:"))
    assert [int(t) for t in line.split()[1:]] == want
    rng = np.random.default_rng(4)
    prompts = [helpers.random_ids(rng, cases.RAW["D"]["vocab"], n) for n in (6, 13, 4)]
    params = [SamplingParams(max_tokens=12, temperature=0.9, top_k=10, seed=7 + i) for i in range(3)]
    together = LLMEngine.from_folder(folder, EngineConfig(block_size=4, num_blocks=64, max_batch_size=4, dtype="float32"))
    got = together.generate(prompts, params)
    for prompt, sp, tokens in zip(prompts, params, got):
        alone = LLMEngine.from_folder(folder, EngineConfig(block_size=16, num_blocks=16, max_batch_size=1, dtype="float32"))
        assert alone.generate([prompt], sp) == [tokens]
