"""A plain, slow implementation of the Gekopel decoder: one function per mechanism, whole sequences
at once on the CPU, no cache and no state carried between calls.  It shares nothing with the engine:
it reads the raw config.json dictionary and a dictionary of tensors by name.

Notation: T tokens of one sequence at positions 0 .. T-1, W the model width, H heads, G key/value
heads, D the query/key size of a head, E its value size, J the taps of a short convolution.
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


def lin(h: torch.Tensor, w: torch.Tensor) -> torch.Tensor:
    """w h for every row of h, w stored [out, in]."""
    return _r(_r(h) @ _r(w).T)


# ---------------------------------------------------------------- norms and activations
def unit_rms(x: torch.Tensor, eps: float) -> torch.Tensor:
    """x / sqrt(mean(x^2) + eps) over the last dimension."""
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)


def rms_norm(x: torch.Tensor, gain: torch.Tensor, eps: float) -> torch.Tensor:
    return unit_rms(x, eps) * gain


def unit_length(x: torch.Tensor) -> torch.Tensor:
    """x / sqrt(sum(x^2) + 1e-6) over the last dimension."""
    return x / torch.sqrt((x * x).sum(dim=-1, keepdim=True) + 1e-6)


def sigmoid(z: torch.Tensor) -> torch.Tensor:
    return 1.0 / (1.0 + torch.exp(-z))


def silu(z: torch.Tensor) -> torch.Tensor:
    return z * sigmoid(z)


def softplus(z: torch.Tensor) -> torch.Tensor:
    """log(1 + exp(z)), without overflow for large z."""
    return torch.clamp(z, min=0.0) + torch.log1p(torch.exp(-z.abs()))


def relu_squared(z: torch.Tensor) -> torch.Tensor:
    return torch.clamp(z, min=0.0) ** 2


# ---------------------------------------------------------------- short convolution
def short_conv(u: torch.Tensor, w: torch.Tensor) -> torch.Tensor:
    """u [T, C], w [C, J]: y_t = sum_j w[:, j] u_(t - J + 1 + j), with zeros before the first token: the
    last column of w multiplies the current token."""
    T, J = u.shape[0], w.shape[1]
    u, w = _r(u), _r(w)
    y = torch.zeros_like(u)
    for j in range(J):
        back = J - 1 - j
        if back < T:
            y[back:] += w[:, j] * u[:T - back]
    return y


# ---------------------------------------------------------------- gated delta rule
def delta_recurrence(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, beta: torch.Tensor, g: torch.Tensor) -> torch.Tensor:
    """q, k [T, G, D], v [T, H, E], beta, g [T, H]; head a reads queries and keys of group a // (H / G).  Per
    head, with S [D, E] zero before the first token: S <- g S, u = beta (v - S^T k), S <- S + k u^T,
    o = S^T q.  Returns o [T, H, E]."""
    T, H, E = v.shape
    G, D = q.shape[1], q.shape[2]
    S = torch.zeros(H, D, E, dtype=DTYPE)
    out = torch.zeros(T, H, E, dtype=DTYPE)
    for t in range(T):
        kt, qt = (x[t].repeat_interleave(H // G, dim=0) for x in (k, q))      # [H, D]
        S = g[t][:, None, None] * S
        u = beta[t][:, None] * (v[t] - torch.einsum("hde,hd->he", S, kt))
        S = S + kt[:, :, None] * u[:, None, :]
        out[t] = torch.einsum("hde,hd->he", S, qt)
    return out


def delta_mixer(h: torch.Tensor, tensors: Dict[str, torch.Tensor], p: str, m: dict, eps: float) -> torch.Tensor:
    """The mixer of a layer of type `delta` (tensors p + q, k, v, their .conv, b, a, A_log, dt_bias, norm, g, o)."""
    T, H, G, D, E = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k, v = (_r(silu(short_conv(lin(h, tensors[p + n]), tensors[p + n + ".conv"]))) for n in ("q", "k", "v"))
    q = unit_length(q.view(T, G, D)) * D ** -0.5
    k = unit_length(k.view(T, G, D))
    beta = sigmoid(lin(h, tensors[p + "b"]))
    g = torch.exp(-torch.exp(tensors[p + "A_log"]) * softplus(lin(h, tensors[p + "a"]) + tensors[p + "dt_bias"]))
    o = delta_recurrence(q, k, v.view(T, H, E), beta, g)
    y = unit_rms(o, eps) * tensors[p + "norm"] * silu(lin(h, tensors[p + "g"])).view(T, H, E)
    return lin(y.reshape(T, H * E), tensors[p + "o"])


# ---------------------------------------------------------------- chunked attention with a distance bias and a sink
def distance_bucket(n: int, buckets: int, bias_max: int) -> int:
    """Row of the bias table for a key n positions back."""
    half = buckets // 2
    if n < half:
        return n
    return min(buckets - 1, half + math.floor(math.log(n / half) / math.log(bias_max / half) * (buckets - half)))


def distance_bias(rel: torch.Tensor, bias_max: int, T: int) -> torch.Tensor:
    """[H, T, T]: rel[bucket(i - j), a] for the key j of the query i (zero for j > i)."""
    rows = torch.tensor([distance_bucket(n, rel.shape[0], bias_max) for n in range(T)])
    i = torch.arange(T)
    dist = (i[:, None] - i[None, :]).clamp(min=0)
    return rel[rows[dist]].permute(2, 0, 1)


def chunk_attention(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, scale: float, bias: torch.Tensor,
                    sink: torch.Tensor, chunk: int) -> torch.Tensor:
    """q [T, H, D], k [T, G, D], v [T, G, E], bias [H, T, T], sink [H]; query head a uses key/value head
    a // (H / G); the query at i sees the keys j <= i of its own chunk (i // chunk == j // chunk; chunk 0:
    every j <= i); the softmax's denominator has one more term exp(sink_a).  Returns [T, H, E]."""
    T, H, _ = q.shape
    G = k.shape[1]
    i = torch.arange(T)
    seen = i[:, None] >= i[None, :]
    if chunk:
        seen &= (i[:, None] // chunk) == (i[None, :] // chunk)
    out = torch.zeros(T, H, v.shape[2], dtype=DTYPE)
    for a in range(H):
        g = a // (H // G)
        s = (q[:, a] @ k[:, g].T) * scale + bias[a]
        s = s.masked_fill(~seen, -math.inf)
        s = torch.cat([s, sink[a].expand(T, 1)], dim=1)
        out[:, a] = _r(torch.softmax(s, dim=-1)[:, :T]) @ v[:, g]
    return out


def attention_mixer(h: torch.Tensor, tensors: Dict[str, torch.Tensor], p: str, m: dict) -> torch.Tensor:
    """The mixer of a layer of type `attention` (tensors p + q, k, v, rel, sink, o)."""
    T, H, G, D, E = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k, v = (lin(h, tensors[p + n]) for n in ("q", "k", "v"))
    bias = distance_bias(tensors[p + "rel"], int(m["bias_max"]), T)
    chunk = int((m.get("mask") or {}).get("size", 0))
    y = _r(chunk_attention(q.view(T, H, D), k.view(T, G, D), v.view(T, G, E), float(m["scale"]), bias,
                           tensors[p + "sink"], chunk))
    return lin(y.reshape(T, H * E), tensors[p + "o"])


# ---------------------------------------------------------------- feed-forwards
def relu2_mlp(h: torch.Tensor, up: torch.Tensor, down: torch.Tensor) -> torch.Tensor:
    return lin(_r(relu_squared(_r(h) @ _r(up).T)), down)


# With ROUTER_GAPS a list, every call of grouped_choice appends one number per token: by how much the router's
# choice is decided.  A test that compares with reduced precision leaves out the tokens whose choice hangs on
# less than that precision can tell.
ROUTER_GAPS: Optional[list] = None


def grouped_choice(scores: torch.Tensor, correction: torch.Tensor, top: int, count: int, keep: int) -> torch.Tensor:
    """scores [T, X] -> the numbers [T, top] of the experts each token uses: those with the largest
    scores + correction among the experts of the `keep` best of `count` equal groups of neighbours, a group's
    rank given by the sum of its two largest."""
    T, X = scores.shape
    choice = scores + correction
    size = X // count
    grouped = torch.sort(choice.view(T, count, size), dim=-1, descending=True).values
    rank = grouped[:, :, :2].sum(dim=-1)                                            # [T, count]
    best = torch.topk(rank, keep, dim=-1).indices
    allowed = torch.zeros(T, count, dtype=torch.bool).scatter_(1, best, True)
    allowed = allowed.repeat_interleave(size, dim=1)
    open_to = choice.masked_fill(~allowed, -math.inf)
    if ROUTER_GAPS is not None:
        srt = torch.sort(open_to, dim=-1, descending=True).values
        gap = srt[:, top - 1] - srt[:, top] if top < X else torch.full((T,), math.inf, dtype=DTYPE)
        if keep < count:
            ranks = torch.sort(rank, dim=-1, descending=True).values
            gap = torch.minimum(gap, ranks[:, keep - 1] - ranks[:, keep])
        ROUTER_GAPS.append(gap)
    return torch.topk(open_to, top, dim=-1).indices


def routed_experts(h: torch.Tensor, tensors: Dict[str, torch.Tensor], p: str, mlp: dict) -> torch.Tensor:
    """Experts relu2_mlp chosen by grouped_choice over s = sigmoid(router h), weighted by s / (sum of the chosen s
    + 1e-20) * router.scale, and a shared one times sigmoid(sg h)."""
    r = mlp["router"]
    n, top = int(r["experts"]), int(r["top"])
    groups = r.get("groups") or {"count": 1, "keep": 1}
    scores = sigmoid(_r(h) @ tensors[p + "router"].T)
    chosen = grouped_choice(scores, tensors[p + "correction"], top, int(groups["count"]), int(groups["keep"]))
    weights = torch.gather(scores, 1, chosen)
    weights = weights / (weights.sum(dim=-1, keepdim=True) + 1e-20) * float(r["scale"])
    out = torch.zeros_like(h)
    for e in range(n):
        for c in range(top):
            rows = (chosen[:, c] == e).nonzero().flatten()
            if rows.numel():
                out[rows] += weights[rows, c][:, None] * relu2_mlp(h[rows], tensors[f"{p}e{e}.up"], tensors[f"{p}e{e}.down"])
    if mlp.get("shared"):
        gate = sigmoid(_r(h) @ tensors[p + "shared.sg"].T)
        out = out + gate * relu2_mlp(h, tensors[p + "shared.up"], tensors[p + "shared.down"])
    return out


# ---------------------------------------------------------------- the model
def layer_forward(x: torch.Tensor, tensors: Dict[str, torch.Tensor], i: int, layer: dict, eps: float) -> torch.Tensor:
    p = f"l{i}."
    h = _r(rms_norm(x, tensors[p + "norm1"], eps))
    if layer["type"] == "delta":
        y = delta_mixer(h, tensors, p + "mix.", layer["mixer"], eps)
    elif layer["type"] == "attention":
        y = attention_mixer(h, tensors, p + "mix.", layer["mixer"])
    else:
        raise ValueError(f"unknown layer type {layer['type']!r}")
    x = x + rms_norm(y, tensors[p + "norm1b"], eps)
    mlp = layer.get("mlp")
    if mlp is not None:
        h = _r(rms_norm(x, tensors[p + "norm2"], eps))
        if mlp["kind"] == "dense":
            y = relu2_mlp(h, tensors[p + "mlp.up"], tensors[p + "mlp.down"])
        elif mlp["kind"] == "moe":
            y = routed_experts(h, tensors, p + "mlp.", mlp)
        else:
            raise ValueError(f"unknown feed-forward {mlp['kind']!r}")
        x = x + rms_norm(y, tensors[p + "norm2b"], eps)
    return x


def forward(cfg: dict, tensors: Dict[str, torch.Tensor], tokens: List[int],
            residuals: Optional[List[torch.Tensor]] = None) -> torch.Tensor:
    """Logits [T, vocab] of one whole sequence.  With `residuals` a list, the residual stream after every
    layer is appended to it."""
    eps = float(cfg["norm"]["eps"])
    x = tensors["embed"][torch.tensor(tokens, dtype=torch.long)].to(DTYPE) * float(cfg["embedding"]["scale"])
    x = x + tensors["pos"][:len(tokens)]
    for i, layer in enumerate(cfg["layers"]):
        x = layer_forward(x, tensors, i, layer, eps)
        if residuals is not None:
            residuals.append(x.clone())
    return lin(_r(rms_norm(x, tensors["final.norm"], eps)), tensors["head"])


def greedy(cfg: dict, tensors: Dict[str, torch.Tensor], prompt: List[int], n_new: int) -> List[int]:
    tokens = list(prompt)
    for _ in range(n_new):
        tokens.append(int(forward(cfg, tensors, tokens)[-1].argmax()))
    return tokens[len(prompt):]
