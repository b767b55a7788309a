"""A plain, slow implementation of the Telapel decoder: one function per mechanism, whole sequences
at once on the CPU, no cache and no state carried between calls.  It shares nothing with the engine:
it reads the raw config.json dictionary and a dictionary of tensors by name.

Notation: T tokens of one sequence at positions 0 .. T-1, W the model width, H heads, G key/value
heads, D the (plain) query/key size of a head, P the rotated size beside it, E its value size, J the taps
of a short convolution, C the channels of a recurrence in B blocks.
"""

from __future__ import annotations

import json
import math
import os
from typing import Dict, List, Optional, Tuple

import torch
from safetensors import safe_open

DTYPE = torch.float64       # what the functions compute in


def read_model_folder(path: str) -> Tuple[dict, Dict[str, torch.Tensor]]:
    with open(os.path.join(path, "config.json"), "r", encoding="utf-8") as fh:
        cfg = json.load(fh)
    tensors: Dict[str, torch.Tensor] = {}
    with safe_open(os.path.join(path, "model.safetensors"), framework="pt", device="cpu") as fh:
        for name in fh.keys():
            t = fh.get_tensor(name)
            tensors[name] = t.to(DTYPE) if t.is_floating_point() else t.to(torch.int64)
    return cfg, tensors


# With ROUNDING set to torch.bfloat16 every matrix product and short convolution takes operands
# rounded to that format and its result is rounded to it too, as a kernel that computes "in bfloat16
# with 32-bit accumulation" does.  The difference between the two modes is the size of what
# rounding alone does to the logits: the tests' bound for the engine's bfloat16 path is a multiple
# of it.
ROUNDING = None


def _r(x: torch.Tensor) -> torch.Tensor:
    return x if ROUNDING is None else x.to(ROUNDING).to(DTYPE)


def lin(h: torch.Tensor, w: torch.Tensor, bias: Optional[torch.Tensor] = None) -> torch.Tensor:
    """w h (+ bias) for every row of h, w stored [out, in]."""
    y = _r(h) @ _r(w).T
    return _r(y if bias is None else y + bias)


# ---------------------------------------------------------------- norms and activations
def rms_norm(x: torch.Tensor, gain: torch.Tensor, eps: float) -> torch.Tensor:
    """x / sqrt(mean(x^2) + eps) * gain over the last dimension."""
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps) * gain


def sigmoid(z: torch.Tensor) -> torch.Tensor:
    return 1.0 / (1.0 + torch.exp(-z))


def softplus(z: torch.Tensor) -> torch.Tensor:
    """log(1 + exp(z)), without overflow for large z."""
    return torch.clamp(z, min=0.0) + torch.log1p(torch.exp(-z.abs()))


def gelu_tanh(z: torch.Tensor) -> torch.Tensor:
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def clamped_swish_unit(gate: torch.Tensor, up: torch.Tensor, limit: float) -> torch.Tensor:
    """g sigmoid(1.702 g) (u + 1) with g = min(gate, limit) and u = up held within -limit .. limit."""
    g, u = torch.clamp(gate, max=limit), torch.clamp(up, min=-limit, max=limit)
    return g * sigmoid(1.702 * g) * (u + 1.0)


# ---------------------------------------------------------------- short convolution
def short_conv(u: torch.Tensor, w: torch.Tensor, bias: Optional[torch.Tensor] = None) -> torch.Tensor:
    """u [T, C], w [C, J]: y[t] = w[:, 0] u[t - J + 1] + ... + w[:, J - 1] u[t] (+ bias), with zeros before the first token: the
    last column of w multiplies the current token."""
    T, J = u.shape[0], w.shape[1]
    u, w = _r(u), _r(w)
    y = torch.zeros_like(u)
    for j in range(J):
        back = J - 1 - j
        if back < T:
            y[back:] += w[:, j] * u[:T - back]
    return y if bias is None else y + bias


# ---------------------------------------------------------------- real-gated linear recurrence
def block_product(u: torch.Tensor, w: torch.Tensor, bias: torch.Tensor) -> torch.Tensor:
    """u [T, C] in B equal parts, w [B, C / B, C / B] stored [out, in], bias [B, C / B]: every part through its own
    square matrix."""
    T = u.shape[0]
    B, size, _ = w.shape
    y = torch.stack([_r(u[:, b * size:(b + 1) * size]) @ _r(w[b]).T + bias[b] for b in range(B)], dim=1)
    return y.reshape(T, B * size)


def gated_recurrence(u: torch.Tensor, r: torch.Tensor, i: torch.Tensor, lam: torch.Tensor) -> torch.Tensor:
    """a = exp(-8 r softplus(lam)); S <- a S + i u sqrt(1 - a^2), S zero before the first token.
    All of [T, C]; returns every S_t."""
    log_a = -8.0 * r * softplus(lam)
    a = torch.exp(log_a)
    x = torch.sqrt(-torch.expm1(2.0 * log_a)) * i * u
    S = torch.zeros(u.shape[1], dtype=DTYPE)
    out = torch.zeros_like(u)
    for t in range(u.shape[0]):
        S = a[t] * S + x[t]
        out[t] = S
    return out


def rglru_mixer(h: torch.Tensor, tensors: Dict[str, torch.Tensor], p: str) -> torch.Tensor:
    """The mixer of a layer of type `rglru` (tensors p + y, x, conv, ra, ri and their .b, lam, o)."""
    y = gelu_tanh(lin(h, tensors[p + "y"], tensors[p + "y.b"]))
    u = _r(short_conv(lin(h, tensors[p + "x"], tensors[p + "x.b"]), tensors[p + "conv"], tensors[p + "conv.b"]))
    r = sigmoid(block_product(u, tensors[p + "ra"], tensors[p + "ra.b"]))
    i = sigmoid(block_product(u, tensors[p + "ri"], tensors[p + "ri.b"]))
    return lin(_r(gated_recurrence(u, r, i, tensors[p + "lam"]) * y), tensors[p + "o"])


# ---------------------------------------------------------------- latent attention
def rotate_pairs(x: torch.Tensor, base: float) -> torch.Tensor:
    """x [T, ..., P]: neighbours (2i, 2i + 1) of the last dimension turned by position * base^(-2i / P)."""
    T, dims = x.shape[0], x.shape[-1]
    f = torch.tensor([float(base) ** (-2.0 * i / dims) for i in range(dims // 2)], dtype=DTYPE)
    a = torch.arange(T, dtype=DTYPE)[:, None] * f
    a = a.view(T, *([1] * (x.dim() - 2)), dims // 2)
    u, v = x[..., 0::2], x[..., 1::2]
    return torch.stack([u * torch.cos(a) - v * torch.sin(a), v * torch.cos(a) + u * torch.sin(a)], dim=-1).reshape(x.shape)


def latent_mixer(h: torch.Tensor, tensors: Dict[str, torch.Tensor], p: str, m: dict, eps: float) -> torch.Tensor:
    """The mixer of a layer of type `latent_attention` (tensors p + dq, dq.norm, uq, dkv, dkv.norm, uk, uv, o)."""
    T, H, D, P, E, R = h.shape[0], m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    cq = rms_norm(lin(h, tensors[p + "dq"]), tensors[p + "dq.norm"], eps)
    q = lin(cq, tensors[p + "uq"]).view(T, H, D + P)
    ckv = lin(h, tensors[p + "dkv"])
    c = _r(rms_norm(ckv[:, :R], tensors[p + "dkv.norm"], eps))
    k_rot = _r(rotate_pairs(ckv[:, R:], m["rot"]["base"]))
    q_rot = _r(rotate_pairs(q[..., D:], m["rot"]["base"]))
    k, v = lin(c, tensors[p + "uk"]).view(T, H, D), lin(c, tensors[p + "uv"]).view(T, H, E)
    i = torch.arange(T)
    later = i[None, :] > i[:, None]
    out = torch.zeros(T, H, E, dtype=DTYPE)
    for a in range(H):
        s = (q[:, a, :D] @ k[:, a].T + q_rot[:, a] @ k_rot.T) * float(m["scale"])
        out[:, a] = _r(torch.softmax(s.masked_fill(later, -math.inf), dim=-1)) @ v[:, a]
    return lin(_r(out.reshape(T, H * E)), tensors[p + "o"])


# ---------------------------------------------------------------- windowed attention with a bias by distance
def slopes(H: int) -> torch.Tensor:
    """2^(-8 (a + 1) / H) for head a."""
    return torch.tensor([2.0 ** (-8.0 * (a + 1) / H) for a in range(H)], dtype=DTYPE)


def query_temperature(T: int, coef: float, every: int) -> torch.Tensor:
    """1 + coef ln(floor((p + 1) / every) + 1) for the positions p = 0 .. T-1."""
    return torch.tensor([1.0 + coef * math.log((p + 1) // every + 1) for p in range(T)], dtype=DTYPE)


def window_attention(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, scale: float, cap: float, slope: torch.Tensor,
                     window: int, sink: Optional[float] = 0.0) -> torch.Tensor:
    """q [T, H, D], k [T, G, D], v [T, G, E]; query head a uses key/value head a // (H / G).  Scores (q . k) scale
    -> cap tanh(. / cap) (cap 0: as they are) -> minus slope_a (i - j); the query at i sees the keys j with
    0 <= i - j < window (window 0: every j <= i); the softmax's denominator has one more term exp(sink) (None: no
    such term).  Returns [T, H, E]."""
    T, H, _ = q.shape
    G = k.shape[1]
    i = torch.arange(T)
    dist = i[:, None] - i[None, :]
    seen = dist >= 0
    if window:
        seen &= dist < window
    out = torch.zeros(T, H, v.shape[2], dtype=DTYPE)
    for a in range(H):
        g = a // (H // G)
        s = (q[:, a] @ k[:, g].T) * scale
        if cap:
            s = cap * torch.tanh(s / cap)
        s = (s - slope[a] * dist).masked_fill(~seen, -math.inf)
        if sink is not None:
            s = torch.cat([s, torch.full((T, 1), float(sink), dtype=DTYPE)], dim=1)
        out[:, a] = _r(torch.softmax(s, dim=-1)[:, :T]) @ v[:, g]
    return out


def attention_mixer(h: torch.Tensor, tensors: Dict[str, torch.Tensor], p: str, m: dict, eps: float) -> torch.Tensor:
    """The mixer of a layer of type `attention` (tensors p + q, k and their .b, .conv, .norm, and o)."""
    T, H, G, D = h.shape[0], m["heads"], m["kv_heads"], m["dim"]
    q, k = (_r(short_conv(lin(h, tensors[p + n], tensors[p + n + ".b"]), tensors[p + n + ".conv"])) for n in ("q", "k"))
    v = k.view(T, G, D)
    qn = rms_norm(q.view(T, H, D), tensors[p + "q.norm"], eps)
    kn = _r(rms_norm(k.view(T, G, D), tensors[p + "k.norm"], eps))
    temp = m.get("q_temp")
    if temp:
        qn = qn * query_temperature(T, float(temp["coef"]), int(temp["every"]))[:, None, None]
    y = window_attention(_r(qn), kn, v, float(m["scale"]), float(m.get("softcap") or 0.0), slopes(H),
                         int((m.get("mask") or {}).get("size") or 0))
    return lin(_r(y.reshape(T, H * D)), tensors[p + "o"])


# ---------------------------------------------------------------- feed-forward
def clamped_mlp(h: torch.Tensor, gate: torch.Tensor, up: torch.Tensor, down: torch.Tensor, limit: float) -> torch.Tensor:
    return lin(_r(clamped_swish_unit(lin(h, gate), lin(h, up), limit)), down)


# With ROUTER_GAPS a list, every call of grouped_choice appends one number per token: by how much the router's
# choice is decided.  A test that compares with reduced precision leaves out the tokens whose choice hangs on
# less than that precision can tell.
ROUTER_GAPS: Optional[list] = None


def grouped_choice(scores: torch.Tensor, top: int, count: int, keep: int) -> torch.Tensor:
    """scores [T, X] -> the numbers [T, top] of the experts each token uses: those with the largest scores among the
    experts of the `keep` best of `count` runs of equal length, a run's rank its largest score."""
    T, X = scores.shape
    size = X // count
    rank = scores.view(T, count, size).max(dim=-1).values                           # [T, count]
    best = torch.topk(rank, keep, dim=-1).indices
    allowed = torch.zeros(T, count, dtype=torch.bool).scatter_(1, best, True).repeat_interleave(size, dim=1)
    open_to = scores.masked_fill(~allowed, -math.inf)
    if ROUTER_GAPS is not None:
        # (of logarithms: by how much the logits differ)
        srt = torch.sort(torch.log(scores).masked_fill(~allowed, -math.inf), dim=-1, descending=True).values
        gap = srt[:, top - 1] - srt[:, top] if top < X else torch.full((T,), math.inf, dtype=DTYPE)
        if keep < count:
            ranks = torch.sort(torch.log(rank), dim=-1, descending=True).values
            gap = torch.minimum(gap, ranks[:, keep - 1] - ranks[:, keep])
        ROUTER_GAPS.append(gap)
    return torch.topk(open_to, top, dim=-1).indices


def routed_experts(h: torch.Tensor, tensors: Dict[str, torch.Tensor], p: str, mlp: dict) -> torch.Tensor:
    """Experts clamped_mlp chosen by grouped_choice over s = softmax(router h), weighted by s / (sum of the chosen s
    + 1e-20), and a shared one with its own limit for every token."""
    r = mlp["router"]
    n, top, limit = int(r["experts"]), int(r["top"]), float(mlp["expert"]["limit"])
    groups = r.get("groups") or {"count": 1, "keep": 1}
    scores = torch.softmax(_r(h) @ tensors[p + "router"].T, dim=-1)
    chosen = grouped_choice(scores, top, int(groups["count"]), int(groups["keep"]))
    weights = torch.gather(scores, 1, chosen)
    weights = weights / (weights.sum(dim=-1, keepdim=True) + 1e-20)
    out = torch.zeros_like(h)
    for e in range(n):
        for c in range(top):
            rows = (chosen[:, c] == e).nonzero().flatten()
            if rows.numel():
                out[rows] += weights[rows, c][:, None] * clamped_mlp(
                    h[rows], *(tensors[f"{p}e{e}.{n_}"] for n_ in ("gate", "up", "down")), limit)
    if mlp.get("shared"):
        out = out + clamped_mlp(h, *(tensors[f"{p}shared.{n_}"] for n_ in ("gate", "up", "down")),
                                float(mlp["shared"]["limit"]))
    return out


# ---------------------------------------------------------------- the model
def layer_forward(x: torch.Tensor, tensors: Dict[str, torch.Tensor], i: int, layer: dict, eps: float) -> torch.Tensor:
    """A layer whose tensors are named l<i>: the sublayers read the residual itself, and their outputs are normed."""
    p, m = f"l{i}.", layer["mixer"]
    if layer["type"] == "rglru":
        y = rglru_mixer(x, tensors, p + "mix.")
    elif layer["type"] == "latent_attention":
        y = latent_mixer(x, tensors, p + "mix.", m, eps)
    elif layer["type"] == "attention":
        y = attention_mixer(x, tensors, p + "mix.", m, eps)
    else:
        raise ValueError(f"unknown layer type {layer['type']!r}")
    x = x + rms_norm(y, tensors[p + "norm1"], eps)
    if layer.get("mlp") is not None:
        x = x + rms_norm(routed_experts(x, tensors, p + "mlp.", layer["mlp"]), tensors[p + "norm2"], eps)
    return x


def forward(cfg: dict, tensors: Dict[str, torch.Tensor], tokens: List[int],
            residuals: Optional[List[torch.Tensor]] = None) -> torch.Tensor:
    """Logits [T, vocab] of one whole sequence.  With `residuals` a list, the residual stream after every
    layer is appended to it."""
    eps = float(cfg["norm"]["eps"])
    x = tensors["embed"][torch.tensor(tokens, dtype=torch.long)].to(DTYPE)
    for i, layer in enumerate(cfg["layers"]):
        named = i
        while cfg["layers"][named].get("weights_of") is not None:
            named = int(cfg["layers"][named]["weights_of"])
        x = layer_forward(x, tensors, named, layer, eps)
        if residuals is not None:
            residuals.append(x.clone())
    return lin(_r(rms_norm(x, tensors["final.norm"], eps)), tensors["embed"])


def greedy(cfg: dict, tensors: Dict[str, torch.Tensor], prompt: List[int], n_new: int) -> List[int]:
    tokens = list(prompt)
    for _ in range(n_new):
        tokens.append(int(forward(cfg, tensors, tokens)[-1].argmax()))
    return tokens[len(prompt):]
