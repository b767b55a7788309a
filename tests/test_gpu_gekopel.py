"""Gekopel on the GPU against the plain implementation (tests/plain_gekopel.py): each new kernel
alone (the gated delta rule in both its forms, token by token and in chunks, with its gate and norm;
chunks, numbers by distance and sinks in every attention kernel; the router with correction and groups;
the weighted sum of the experts' outputs with a gated shared one; the squared relu as an epilogue of every
product kernel; the scaled embedding with positions); whole prompts against token-by-token decoding,
portions down to two tokens and mixed batches with pages, request slots and states used again, steps
that want no logits, in 32-bit and bfloat16; long decoding; configurations drawn at random; greedy
generation through LLMEngine."""

import json
import math
import os
import subprocess
import sys
import types

import numpy as np
import pytest
import torch

import gekopel_cases as cases
import helpers
import plain_gekopel as P
from mini_gpt_inference_amd import EngineConfig, SamplingParams
from mini_gpt_inference_amd.engine.llm_engine import LLMEngine
from mini_gpt_inference_amd.engine.replay import TraceError, TraceReplayer
from mini_gpt_inference_amd.ops import kernels
from mini_gpt_inference_amd.ops.linear import linear
from mini_gpt_inference_amd.parts.base import Workspace
from mini_gpt_inference_amd.parts.mixers import distance_buckets

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
WHOLE = [[(0, 0, 70), (1, 0, 1), (2, 0, 32), (3, 0, 33)]]
PORTIONS = [[(0, 0, 31), (3, 0, 2)], [(0, 31, 2), (1, 0, 1), (3, 2, 30)], [(3, 32, 1), (0, 33, 36), (2, 0, 17)],
            [(0, 69, 1), (2, 17, 15)]]
ONE_BY_ONE = [[(r, t, 1) for r, n in enumerate((70, 1, 32, 33)) if t < n] for t in range(70)]
STARTS, COUNTS = [0, 70, 71, 103], [70, 1, 32, 33]
N_ROWS = 136


def _step_arrays(step):
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


# ---------------------------------------------------------------- the gated delta rule
def _delta_case(H, G, D, E, dtype, seed, kind="plain"):
    """Rows as the mixer lays them out, and the plain result for the four requests.  kind "alike": keys of
    one direction with hardly any noise and step sizes near one, so that every token takes back most of what the
    one before wrote; "extreme": heads in which decays of nearly 1 and of e^-60 follow each other."""
    g = torch.Generator().manual_seed(seed)
    x = _rnd(g, N_ROWS, 2 * G * D + H * E + 3, dtype=dtype)
    z = _rnd(g, N_ROWS, 2 * H + H * E + 5, dtype=dtype, scale=2.0)
    dt_bias, a_log, norm = _rnd(g, H) - 2.0, _rnd(g, H), 1.0 + 0.1 * _rnd(g, E)
    if kind == "alike":
        x[:, G * D:2 * G * D] = (1.0 + 0.05 * _rnd(g, N_ROWS, G * D)).to(TDT[dtype])
        z[:, 2:2 + H] = 6.0
        dt_bias -= 6.0
    if kind == "extreme":
        z[:, 2 + H:2 + 2 * H] = torch.where(torch.rand(N_ROWS, H, generator=g) < 0.3, 60.0, -8.0).to(TDT[dtype])
        a_log[:] = 0.0
    offs = dict(q_off=0, k_off=G * D, v_off=2 * G * D, b_off=2, a_off=2 + H, gate_off=2 + 2 * H)
    want = torch.zeros(N_ROWS, H, E, dtype=P.DTYPE)
    for s, c in zip(STARTS, COUNTS):
        rows, logits = _d(x[s:s + c]), _d(z[s:s + c])
        q = P.unit_length(rows[:, :G * D].view(c, G, D)) * D ** -0.5
        k = P.unit_length(rows[:, G * D:2 * G * D].view(c, G, D))
        v = rows[:, 2 * G * D:2 * G * D + H * E].view(c, H, E)
        beta = P.sigmoid(logits[:, 2:2 + H])
        decay = torch.exp(-torch.exp(_d(a_log)) * P.softplus(logits[:, 2 + H:2 + 2 * H] + _d(dt_bias)))
        want[s:s + c] = P.delta_recurrence(q, k, v, beta, decay)
    gate = P.silu(_d(z[:, 2 + 2 * H:2 + 2 * H + H * E])).view(N_ROWS, H, E)
    gated = P.unit_rms(want, 1e-5) * _d(norm) * gate
    return (x, z, offs, dict(dt_bias=dt_bias.to(DEV), a_log=a_log.to(DEV)), norm.to(DEV), want.reshape(N_ROWS, H * E),
            gated.reshape(N_ROWS, H * E))


def _run_delta(plan, chunked, H, G, D, E, case, state, gated=False):
    x, z, offs, consts, norm = case[:5]
    got = torch.zeros(N_ROWS, H * E, dtype=P.DTYPE)
    for step in plan:
        rows, cu, pos, _, slots = _step_arrays(step)
        n, n_req = len(rows), len(step) + 1
        xs, zs = x[rows].to(DEV), z[rows].to(DEV)
        out = torch.full((n + 1, H * E), 9.0, device=DEV, dtype=x.dtype if gated else torch.float32)
        args = (xs, offs["q_off"], offs["k_off"], offs["v_off"], zs, offs["b_off"], offs["a_off"], H, G, D, E, consts["dt_bias"],
                consts["a_log"], state, slots, cu, n_req, pos)
        if chunked:
            images = torch.full((kernels.delta_image_floats(n, n_req, H, D),), float("nan"), device=DEV)
            assert kernels.delta_state_chunked(*args, images, out, n, q_scale=D ** -0.5)
        elif gated:
            kernels.delta_state(*args, out, n, q_scale=D ** -0.5, gate_off=offs["gate_off"], norm_weight=norm, eps=1e-5)
        else:
            kernels.delta_state(*args, out, n, q_scale=D ** -0.5)
        assert (out[n] == 9.0).all()
        got[rows] = out[:n].cpu().to(P.DTYPE)
    return got


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("H,G,D,E,kind", [
    (2, 2, 16, 24, "plain"), (6, 2, 20, 12, "plain"), (1, 1, 64, 64, "plain"), (2, 1, 128, 128, "plain"), (3, 3, 12, 130, "plain"),
    (16, 4, 8, 256, "plain"), (4, 1, 40, 20, "plain"), (5, 1, 100, 33, "plain"), (2, 1, 32, 16, "alike"), (2, 2, 64, 32, "alike"),
    (3, 1, 16, 16, "extreme"), (2, 2, 128, 48, "extreme")])
def test_gated_delta_rule(dtype, H, G, D, E, kind):
    """Token by token and in chunks: whole requests of 70, 1, 32 and 33 tokens, the same in portions whose cuts fall
    inside, at and one token beside a chunk's border, and one token a step; then the token-by-token kernel
    goes on from the state the chunked one left, with gate and norm.  States start as NaN and are compared too."""
    case = _delta_case(H, G, D, E, dtype, H * D + E, kind)
    want, gated = case[5:]
    width = H * D * E
    states = {}
    for chunked in (False, True):
        for name, plan in (("whole", WHOLE), ("portions", PORTIONS), ("one by one", ONE_BY_ONE)):
            pool = torch.full((6, width + 5), float("nan"), device=DEV)      # the state is a view of a wider pool's columns
            state = pool[:, :width]
            got = _run_delta(plan, chunked, H, G, D, E, case, state)
            helpers.assert_close(got, want, "float32", f"chunked {chunked} {name}")
            assert torch.isnan(pool[0]).all() and torch.isnan(pool[5]).all() and torch.isnan(pool[:, width:]).all()
            assert torch.isfinite(state[1:5]).all()
            states[(chunked, name)] = state[1:5].cpu()
    ref = states[(False, "whole")]
    for key, st in states.items():
        helpers.assert_close(st, ref, "float32", f"state {key}")
    # chunks first, then single tokens
    pool = torch.full((6, width), float("nan"), device=DEV)
    head = [[(0, 0, 37), (2, 0, 30), (3, 0, 32)]]
    tail = [[(r, t, 1) for r, first, n in ((0, 37, 70), (1, 0, 1), (2, 30, 32), (3, 32, 33)) if first <= t < n] for t in range(70)]
    got = _run_delta(head, True, H, G, D, E, case, pool)
    got2 = _run_delta([s for s in tail if s], False, H, G, D, E, case, pool, gated=True)
    done = torch.zeros(N_ROWS, dtype=torch.bool)
    for r, n in ((0, 37), (2, 30), (3, 32)):
        done[STARTS[r]:STARTS[r] + n] = True
    helpers.assert_close(got[done], want[done], "float32", "chunks")
    helpers.assert_close(got2[~done], gated[~done], dtype, "token by token behind chunks, gate and norm inside")
    pool.fill_(float("nan"))
    helpers.assert_close(_run_delta(WHOLE, False, H, G, D, E, case, pool, gated=True), gated, dtype, "gate and norm inside")


def test_delta_heads_larger_than_the_chunked_form_takes():
    """Head sizes over 128: the chunked form says no and launches nothing, the token-by-token kernel takes them."""
    H, G, D, E = 2, 1, 160, 24
    case = _delta_case(H, G, D, E, "float32", 3)
    assert kernels.delta_image_floats(10, 2, H, D) == 0
    state = torch.full((6, H * D * E), float("nan"), device=DEV)
    helpers.assert_close(_run_delta(PORTIONS, False, H, G, D, E, case, state), case[5], "float32", "heads of 160")


@pytest.mark.parametrize("chunked", [False, True])
def test_a_write_far_back_matters(chunked):
    """With decays near one and small steps the first token's value is still in the output after hundreds of tokens
    (a lost or restarted state shows); a later token with the same key takes it back.  Prompt of 330 tokens in
    portions, then 70 tokens one by one."""
    g = torch.Generator().manual_seed(5)
    T, H, D, E = 400, 2, 32, 16
    x = _rnd(g, T, 2 * D + H * E)
    mark = torch.zeros(D)
    mark[0] = 40.0
    x[:, D] = 0.0                                  # no other key has a share in the marked direction
    x[0, D:2 * D] = mark
    x[0, 2 * D:] *= 30.0
    x[300:, :D] = mark                             # queries for it from token 300 on
    x[360, D:2 * D] = mark                         # written over at token 360
    z = torch.cat([torch.full((T, H), 1.0), torch.full((T, H), -6.0)], dim=1)
    z[0, :H], z[360, :H] = 9.0, 9.0
    dt_bias, a_log = torch.full((H,), -3.0), torch.zeros(H)
    q, k = P.unit_length(_d(x[:, :D])).view(T, 1, D), P.unit_length(_d(x[:, D:2 * D])).view(T, 1, D)
    v, beta = _d(x[:, 2 * D:]).view(T, H, E), P.sigmoid(_d(z[:, :H]))
    decay = torch.exp(-P.softplus(_d(z[:, H:]) + _d(dt_bias)))
    want = P.delta_recurrence(q, k, v, beta, decay)
    assert float(want[359].abs().max()) > 10.0 and float(want[361].abs().max()) < 5.0
    state = torch.full((3, H * D * E), float("nan"), device=DEV)
    got = torch.zeros(T, H * E, dtype=P.DTYPE)
    cuts = [0, 100, 102, 197, 330] + list(range(331, T + 1))
    for first, last in zip(cuts[:-1], cuts[1:]):
        n = last - first
        out = torch.zeros(n, H * E, device=DEV)
        args = (x[first:last].to(DEV), 0, D, 2 * D, z[first:last].to(DEV), 0, H, H, 1, D, E, dt_bias.to(DEV), a_log.to(DEV), state,
                _i32([1]), _i32([0, n]), 1, _i32(list(range(first, last))))
        if chunked and n > 1:
            assert kernels.delta_state_chunked(*args, torch.zeros(kernels.delta_image_floats(n, 1, H, D), device=DEV), out, n)
        else:
            kernels.delta_state(*args, out, n)
        got[first:last] = out.cpu().to(P.DTYPE)
    helpers.assert_close(got, want.reshape(T, H * E), "float32", "a value 359 tokens back")


# ---------------------------------------------------------------- chunks, numbers by distance and sinks in the attention kernels
def _paged(k, v, page, perm, dtype):
    T, G, D = k.shape
    E = v.shape[2]
    kp = torch.full((len(perm), G, page, D), float("nan"), dtype=TDT[dtype])
    vp = torch.full((len(perm), G, page, E), float("nan"), dtype=TDT[dtype])
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
@pytest.mark.parametrize("chunk,T", [(1, 40), (2, 77), (16, 209), (17, 205), (70, 208), (100, 201), (130, 262), (200, 200), (300, 210)])
def test_a_key_just_inside_and_just_outside_the_chunk(dtype, D, chunk, T):
    """The last query is made to look like one key, scaled so that this key takes nearly all the weight if it is
    seen: once the key is the chunk's first, once the one before it."""
    H, G, scale = 4, 2, D ** -0.5
    start = (T - 1) // chunk * chunk
    for far in (start, start - 1):
        if far < 0:
            continue
        g = torch.Generator().manual_seed(7 + D + chunk)
        q, k, v = _rnd(g, T, H, D, dtype=dtype), _rnd(g, T, G, D, dtype=dtype), _rnd(g, T, G, D, dtype=dtype)
        k[far] *= 4.0
        q[-1] = k[far].float().repeat_interleave(H // G, dim=0).to(TDT[dtype])
        none, sink = torch.zeros(H, T, T, dtype=P.DTYPE), torch.full((H,), -1.5, dtype=P.DTYPE)
        want = P.chunk_attention(_d(q), _d(k), _d(v), scale, none, sink, chunk)
        if far < start:
            seen = P.chunk_attention(_d(q), _d(k), _d(v), scale, none, sink, 0)
            assert float((want[-1] - seen[-1]).abs().max()) > 0.3      # without the chunk the key would take over
        _every_attention_kernel(q, k, v, want, dtype, scale, min(100, T // 2), 16, f"chunk {chunk}, key {far} of {T}", window=chunk,
                                chunked=True, sinks=sink.float().to(DEV))


@pytest.mark.parametrize("dtype,D", KERNEL_DIMS)
@pytest.mark.parametrize("buckets,bias_max,chunk", [(16, 40, 0), (32, 200, 0), (2, 5, 0), (32, 90, 110), (8, 300, 64)])
def test_numbers_by_distance(dtype, D, buckets, bias_max, chunk):
    """One bucket of the table stands out per head (an early one, the last of one distance, the first of several,
    the last bucket), so that a number taken one distance off shows; with and without chunks, with sinks of
    very different sizes."""
    T, H, G, scale, page = 233, 4, 2, D ** -0.5, 16
    g = torch.Generator().manual_seed(buckets + bias_max + D)
    q, k, v = _rnd(g, T, H, D, dtype=dtype, scale=0.5), _rnd(g, T, G, D, dtype=dtype, scale=0.5), _rnd(g, T, G, D, dtype=dtype)
    rel = _rnd(g, buckets, H)
    half = buckets // 2
    for a, row in enumerate((min(3, buckets - 1), max(half - 1, 0), min(half, buckets - 1), buckets - 1)):
        rel[row, a] += 6.0
    sink = torch.tensor([-20.0, 0.5, 4.0, 9.0])
    want = P.chunk_attention(_d(q), _d(k), _d(v), scale, P.distance_bias(_d(rel), bias_max, T), _d(sink), chunk)
    table = rel[torch.tensor(distance_buckets(buckets, bias_max))].t().contiguous().to(DEV)
    for first in (0, 100, T - 3):
        _every_attention_kernel(q, k, v, want, dtype, scale, first, page, f"{buckets} buckets to {bias_max}, from {first}",
                                window=chunk, chunked=bool(chunk), sinks=sink.to(DEV), dist_bias=table)


def test_numbers_by_distance_in_steps_of_several_requests():
    """Portions of different lengths on top of different contexts in one launch of the tile kernel, and single tokens
    of different lengths in one launch of the decode kernel."""
    dtype, D, H, G, page, chunk, scale = "bfloat16", 64, 3, 1, 16, 48, 0.125
    g = torch.Generator().manual_seed(3)
    lens, new = [70, 33, 200, 1, 97], [70, 2, 130, 1, 1]
    rel, sink = _rnd(g, 12, H, scale=2.0), _rnd(g, H)
    table = rel[torch.tensor(distance_buckets(12, 30))].t().contiguous().to(DEV)
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
        want = P.chunk_attention(_d(q), _d(k), _d(v), scale, P.distance_bias(_d(rel), 30, T), _d(sink), chunk)
        qs.append(q)
        wants.append(want)
    kp, vp, bt = kp.to(DEV), vp.to(DEV), bt.to(DEV)
    mask = dict(window=chunk, chunked=True, sinks=sink.to(DEV), dist_bias=table)
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


# ---------------------------------------------------------------- the router, the experts' sum, the squared relu, the embedding
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("n,width,experts,top,groups,shared", [
    (9, 40, 6, 2, (3, 2), True), (70, 264, 12, 3, (4, 1), False), (5, 2048, 8, 2, (8, 5), True), (4, 24, 3, 3, (1, 1), True),
    (33, 136, 64, 4, (8, 4), True), (3, 100, 130, 2, (65, 3), False), (2, 4100, 9, 2, (3, 3), True), (6, 64, 256, 8, (8, 2), True)])
def test_router_with_correction_and_groups(dtype, n, width, experts, top, groups, shared):
    g = torch.Generator().manual_seed(n + experts)
    h = _rnd(g, n + 1, width + 8, dtype=dtype)
    w, sg = _rnd(g, experts, width, dtype=dtype, scale=width ** -0.5 * 2.0), _rnd(g, 1, width, dtype=dtype, scale=width ** -0.5 * 2.0)
    correction = _rnd(g, experts, scale=0.5) - 1.2          # most choice scores are negative
    rows = _d(h[:n, :width])
    scores = P.sigmoid(rows @ _d(w).T)
    P.ROUTER_GAPS = []
    try:
        want = P.grouped_choice(scores, _d(correction), top, *groups)
        firm = P.ROUTER_GAPS[0] > 1e-5
    finally:
        P.ROUTER_GAPS = None
    assert int(firm.sum()) >= n - 1
    weights = torch.gather(scores, 1, want)
    weights = weights / (weights.sum(dim=1, keepdim=True) + 1e-20) * 1.75
    chosen = torch.full((n + 1, top), -7, dtype=torch.int32, device=DEV)
    weight, gate = torch.full((n + 1, top), -7.0, device=DEV), torch.full((n + 1,), -7.0, device=DEV)
    kernels.router_topk(h.to(DEV), w.to(DEV), n, top, chosen, weight, correction=correction.to(DEV), groups=groups, normalise=True,
                        scale=1.75, extra=sg.to(DEV) if shared else None, extra_out=gate if shared else None)
    assert (chosen[n] == -7).all() and (weight[n] == -7.0).all() and gate[n] == -7.0
    assert torch.equal(chosen[:n].cpu().long()[firm], want[firm])
    helpers.assert_close(weight[:n].cpu()[firm], weights[firm], "float32", "weights")
    if shared:
        helpers.assert_close(gate[:n], P.sigmoid(rows @ _d(sg).T)[:, 0], "float32", "the shared expert's number")
    # plain scores, scaled, not normalised
    kernels.router_topk(h.to(DEV), w.to(DEV), n, top, chosen, weight, scale=0.5)
    helpers.assert_close(weight[:n], 0.5 * torch.topk(scores, top, dim=1).values, "float32", "scaled scores")


@pytest.mark.parametrize("n,width,top", [(1, 64, 2), (7, 30, 3), (65, 264, 1)])
def test_the_experts_weighted_sum_and_a_gated_row_beside_it(n, width, top):
    g = torch.Generator().manual_seed(n)
    pair_out, y0 = _rnd(g, n * top + 3, width), _rnd(g, n + 1, width)
    pair_weight, extra, gate = torch.rand(n * top, generator=g), _rnd(g, n, width), torch.rand(n, generator=g)
    slots = torch.randperm(n * top + 3, generator=g)[:n * top].to(torch.int32)
    for use_slots in (False, True):
        rows = _d(pair_out)[slots.long()] if use_slots else _d(pair_out)[:n * top]
        want = _d(y0).clone()
        want[:n] += 0.5 * (rows * _d(pair_weight)[:, None]).view(n, top, width).sum(1) + _d(gate)[:, None] * _d(extra)
        y = y0.to(DEV)
        kernels.expert_combine(pair_out.to(DEV), y, n, top, 0.5, pair_slot=slots.to(DEV) if use_slots else None,
                               pair_weight=pair_weight.to(DEV), extra=extra.to(DEV), extra_gate=gate.to(DEV))
        helpers.assert_close(y, want, "float32", "weighted sum")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("n", [1, 5, 16, 33, 64, 70, 300])
@pytest.mark.parametrize("out,inn", [(96, 64), (200, 512), (40, 20), (128, 4096), (1024, 256), (4608, 1536)])
def test_squared_relu_epilogue(dtype, n, out, inn):
    """Through ops.linear, whose choice of kernel goes by the size (decode kernels with and without a split inner size,
    tiled kernel, general kernel)."""
    g = torch.Generator().manual_seed(out + n)
    a, w = _rnd(g, n, inn, dtype=dtype), _rnd(g, out, inn, dtype=dtype, scale=inn ** -0.5)
    ctx = types.SimpleNamespace(exact=dtype == "float32", dtype=TDT[dtype], workspace=Workspace(torch.device(DEV)), n_rows=n,
                                pending=None, copy_budget=None)
    got = torch.full((n + 1, out), 9.0, dtype=TDT[dtype], device=DEV)
    linear(ctx, a.to(DEV), w.to(DEV), None, got[:n], n, kernels.EPI_RELU2)
    assert (got[n] == 9.0).all()
    want = P.relu_squared(_d(a) @ _d(w).T)
    assert float(want.max()) > 1.0 and float((want == 0).double().mean()) > 0.3
    helpers.assert_close(got[:n], want, dtype, "squared relu")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("n,experts,top,width,hidden", [(3, 4, 2, 64, 48), (40, 5, 1, 40, 20), (300, 3, 2, 128, 64), (400, 6, 2, 256, 272)])
def test_grouped_products_with_the_squared_relu(dtype, n, experts, top, width, hidden):
    """Every tile size that a step of this many pairs may come in."""
    g = torch.Generator().manual_seed(n)
    h, w = _rnd(g, n, width, dtype=dtype), _rnd(g, experts, hidden, width, dtype=dtype, scale=width ** -0.5)
    table = torch.stack([torch.randperm(experts, generator=g)[:top] for _ in range(n)]).to(torch.int32)
    want = P.relu_squared(torch.einsum("nw,efw->nef", _d(h), _d(w)))
    for tile in (16, 64, 256):
        slots = kernels.expert_slots(n, top, experts, tile)
        st, sp, te = (torch.zeros(k, dtype=torch.int32, device=DEV) for k in (slots, slots, slots // tile))
        kernels.expert_route(None, None, table.to(DEV), n, experts, st, sp, te, tile)
        out = torch.zeros(slots, hidden, dtype=TDT[dtype], device=DEV)
        if tile == 256:
            if dtype != "bfloat16" or width % 16 or hidden % 16:
                continue
            rows = torch.zeros(slots, width, dtype=TDT[dtype], device=DEV)
            assert kernels.gather_rows(h.to(DEV), st, rows, slots)
            assert kernels.grouped_linear_tiled(rows, w.to(DEV), te, st, out, slots, kernels.EPI_RELU2)
        else:
            kernels.grouped_linear(h.to(DEV), st, w.to(DEV), te, st, out, None, slots, tile, dtype == "bfloat16", kernels.EPI_RELU2)
        st, sp = st.cpu(), sp.cpu()
        used = (st >= 0).nonzero().flatten()
        assert len(used) == n * top
        ref = torch.stack([want[st[s], table[st[s], sp[s] % top]] for s in used.tolist()])
        helpers.assert_close(out[used.to(DEV)], ref, dtype, f"tiles of {tile}")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_scaled_embedding_with_positions(dtype):
    g = torch.Generator().manual_seed(1)
    tok, pos = _rnd(g, 19, 70, dtype=dtype), _rnd(g, 50, 70, dtype=dtype)
    ids, at = torch.randint(0, 19, (9,), generator=g), torch.randint(0, 50, (9,), generator=g)
    x = torch.full((10, 140), 9.0, device=DEV)
    kernels.embed_scaled(_i32(ids.tolist()), tok.to(DEV), x, 9, 3.25, copies=2, positions=_i32(at.tolist()), pos_table=pos.to(DEV))
    want = _d(tok)[ids] * 3.25 + _d(pos)[at]
    helpers.assert_close(x[:9], torch.cat([want, want], dim=1), "float32", "scaled rows with positions")
    assert (x[9] == 9.0).all()


# ---------------------------------------------------------------- the model through the step function
LENGTHS = {"A": [5, 70, 23, 41, 2, 64, 37], "B": [1, 9, 33, 17, 110], "C": [40, 3, 64, 21], "D": [75, 12, 30, 6, 49],
           "E": [33, 4, 70, 18, 2], "F": [130, 1, 66, 40, 9]}
_folders, _plain, _twin = {}, {}, {}


def _folder(tmp_path_factory, name):
    if name not in _folders:
        _folders[name] = cases.write_model(str(tmp_path_factory.mktemp("gekopel") / name), name)
    return _folders[name]


FIRM_GAP = 0.03     # in a router's choice scores: a choice decided by less is no test of reduced precision


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
                bound = 5e-5 * max(1.0, float(np.abs(ref).max())) if dtype == "float32" else 0.1
                assert np.isfinite(row).all() and err <= bound, f"{name} {dtype} {way} {rid} position {pos}: {err:.3e}"


@pytest.mark.parametrize("seed", range(8))
def test_random_configurations(tmp_path, seed):
    """Configurations drawn at random (tests/gekopel_cases.py: random_raw), five requests of lengths
    1 to 200 each, whole, in portions and mixed, in both dtypes.  bfloat16: a position may be one and
    a half times over three times what rounding alone does, the mean may not; a request is compared up to
    its first position where a router's choice is a close call."""
    rng = np.random.default_rng(4000 + seed)
    raw, buckets = cases.random_raw(rng)
    folder = cases.write_raw_model(str(tmp_path / "m"), raw, seed, buckets=buckets)
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
    convolution inputs are carried over hundreds of steps, chunks of both sizes begin and end among
    decoded tokens, the decode steps come from graphs."""
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
def test_sharp_attention_at_chunk_edges_prefill_and_decoding(tmp_path, dtype):
    """Configuration A with the queries and keys of its attention layers scaled up (a sharp softmax) and the
    bias rows spread out: 90 tokens whole, in portions, and with the last 60 one by one, so that chunks of both
    sizes (7 and 37 positions) begin and end among prompt tokens and among decoded ones."""
    def edit(tensors):
        for layer in (0, 2):
            for n in ("q", "k"):
                tensors[f"l{layer}.mix.{n}"] *= 3.0
            tensors[f"l{layer}.mix.rel"] *= 4.0
    folder = cases.write_model(str(tmp_path / "sharp"), "A", edit=edit)
    cfg, w = P.read_model_folder(folder)
    ids = _firm_ids(cfg, w, np.random.default_rng(11), cases.RAW["A"]["vocab"], 90)
    want = P.forward(cfg, w, ids).numpy()
    # the chunk matters: one position less and the logits move
    shorter = json.loads(json.dumps(cfg))
    shorter["layers"][2]["mixer"]["mask"]["size"] -= 1
    assert _row_errors(P.forward(shorter, w, ids).numpy(), want)[40:].max() > 1e-2
    for way, plan in (("whole", helpers.plan_whole({"a": ids})), ("portions", helpers.plan_portions({"a": ids}, None)),
                      ("tail", helpers.plan_tail({"a": ids}, tail=60))):
        replayer = TraceReplayer(folder, dtype, 128, page_size=16, max_live=4, poison=True)
        got = plan.assemble(helpers.run_plan_in_process(replayer, plan), {"a": len(ids)}, cases.RAW["A"]["vocab"])
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


def test_positions_beyond_the_table_are_refused(tmp_path_factory):
    folder = _folder(tmp_path_factory, "C")
    last = cases.RAW["C"]["max_positions"]
    ids = helpers.random_ids(np.random.default_rng(1), cases.RAW["C"]["vocab"], last)
    replayer = TraceReplayer(folder, "float32", 192, page_size=16, max_live=4)
    cfg, w = P.read_model_folder(folder)
    got = replayer.run_step({"step": 0, "entries": [{"id": "a", "tokens": ids, "want": [last - 1]}], "end": []})
    want = P.forward(cfg, w, ids).numpy()[-1:]
    assert _row_errors(got.cpu().numpy(), want).max() <= 5e-5 * max(1.0, float(np.abs(want).max()))
    with pytest.raises((TraceError, ValueError)):
        replayer.run_step({"step": 1, "entries": [{"id": "a", "tokens": [1], "want": [0]}], "end": []})


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
    assert checked >= 6


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
    """`python -m mini_gpt_inference_amd.generate` on a Gekopel folder: the architecture is found by config.json,
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
    assert "Gekopel" in proc.stdout
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
