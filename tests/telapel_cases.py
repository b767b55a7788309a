"""Small Telapel configurations and model folders with random weights for the tests.

The configurations differ from each other in every size and option: the order of the layer types, layers that use
another's tensors (one after the other, and one that uses those of a layer that uses another's), widths that are
and are not multiples of 16, recurrences in one block and in several, of block sizes that the matrix-core kernels take and
that they do not, one to six taps, one head and several, one key/value head, a few and as many as heads, windows of
one position up to longer than any request and none, caps and none, temperatures that change every token, never within a
request and none, latents whose cached rows are below, at and beyond the sizes of the matrix-core kernels, values
smaller and larger than the latent, routed feed-forwards and none, one to four experts a token out of two to twelve, one
group, all groups kept and some left out, groups of one expert, a shared expert with another limit or none."""

from __future__ import annotations

import os
from typing import Callable, Dict, Optional

import torch
from safetensors.torch import save_file

from mini_gpt_inference_amd.config.model_config import write_config_json
from mini_gpt_inference_amd.models import telapel
from mini_gpt_inference_amd.weights.random_init import random_tensors


def rglru(width, blocks, conv):
    return "rglru", {"width": width, "blocks": blocks, "conv": conv}


def latent(heads, dim, rot_dim, vdim, q_rank, kv_rank, scale, base):
    return "latent_attention", {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "q_rank": q_rank, "kv_rank": kv_rank,
                                "scale": scale, "rot": {"base": base, "dims": rot_dim}}


def attention(heads, kv_heads, dim, scale, conv, softcap=None, window=None, temp=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "scale": scale, "conv": conv}
    if softcap:
        m["softcap"] = softcap
    if window:
        m["mask"] = {"size": window}
    if temp:
        m["q_temp"] = {"coef": temp[0], "every": temp[1]}
    return "attention", m


def moe(experts, top, ff, limit, groups=(1, 1), shared=None):
    out = {"kind": "moe", "router": {"experts": experts, "top": top, "groups": {"count": groups[0], "keep": groups[1]}},
           "expert": {"ff": ff, "limit": limit}}
    if shared:
        out["shared"] = {"ff": shared[0], "limit": shared[1]}
    return out


def layer(mixer, mlp, weights_of=None):
    out = {"type": mixer[0], "mixer": mixer[1], "mlp": mlp}
    if weights_of is not None:
        out["weights_of"] = weights_of
    return out


def model(vocab, width, eps, layers):
    return {"architecture": "Telapel", "vocab": vocab, "width": width, "norm": {"eps": eps}, "layers": layers}


_R, _A, _L = rglru(48, 3, 3), attention(6, 2, 24, 0.3, 2, 5.0, 7, (0.5, 3)), latent(3, 12, 8, 20, 40, 24, 0.25, 500.0)
_M = moe(6, 2, 32, 1.0, (3, 2), (40, 0.5))

RAW: Dict[str, dict] = {
    # all three mixers; a window shorter than a page; a layer of each type used twice, one three times
    "A": model(131, 64, 1e-5, [
        layer(_R, _M), layer(_A, None), layer(_L, moe(4, 1, 48, 0.7)), layer(_R, _M, 0), layer(_A, None, 1),
        layer(_L, moe(4, 1, 48, 0.7), 2), layer(_R, _M, 3)]),
    # head sizes and rows that the bfloat16 matrix-core kernels take (64 and 128; a cached row of 64), as many key/value
    # heads as heads, no window, no cap, no temperature; blocks of 32 and of 144; groups of one expert, none shared
    "B": model(77, 96, 1e-6, [
        layer(attention(2, 2, 64, 0.125, 4), moe(5, 2, 64, 1.5, (5, 3))),
        layer(rglru(64, 2, 5), moe(9, 3, 40, 0.8, (3, 3), (72, 2.0))),
        layer(latent(2, 40, 16, 56, 72, 48, 0.15, 1e4), None),
        layer(attention(4, 2, 128, 0.09, 3, 20.0, 50, (0.3, 16)), moe(5, 2, 64, 1.5, (5, 3))),
        layer(rglru(288, 2, 2), None)]),
    # a width, heads and blocks that only the general kernels take; one tap everywhere, a window of one position (a token
    # sees itself only), a temperature that changes at every token, every expert chosen
    "C": model(59, 40, 1e-4, [
        layer(attention(3, 1, 20, 0.6, 1, 2.0, 1, (1.0, 1)), moe(2, 2, 24, 0.6, (1, 1), (24, 1.2))),
        layer(rglru(36, 3, 1), moe(8, 3, 72, 1.1, (2, 1))),
        layer(latent(1, 4, 6, 12, 20, 10, 0.5, 50.0), None),
        layer(attention(4, 4, 12, 0.5, 6, None, 16), None)]),
    # one layer of each, a window that is no multiple of anything
    "D": model(33, 32, 1e-5, [
        layer(latent(2, 8, 8, 16, 24, 16, 0.3, 100.0), moe(6, 2, 16, 1.0, (2, 2), (16, 1.0))),
        layer(attention(2, 1, 16, 0.25, 4, 8.0, 33, (0.4, 10)), moe(4, 2, 16, 0.9, (4, 2))),
        layer(rglru(16, 1, 4), moe(6, 2, 16, 1.0, (2, 2), (16, 1.0)))]),
    # recurrences only: no keys and values, no pages with anything in them
    "E": model(45, 48, 1e-5, [
        layer(rglru(80, 5, 4), moe(4, 2, 24, 1.0, (4, 2), (24, 0.8))), layer(rglru(32, 1, 2), None),
        layer(rglru(32, 1, 2), None, 1)]),
    # attention of both kinds only, with different windows and none, several cached rows (one beyond 128)
    "F": model(64, 80, 1e-5, [
        layer(attention(4, 2, 32, 0.18, 3, 15.0, 40, (0.2, 64)), moe(7, 1, 40, 1.3, (7, 4), (24, 1.3))),
        layer(latent(4, 24, 32, 16, 48, 96, 0.15, 2000.0), None),
        layer(attention(6, 2, 24, 0.2, 2, 4.0, 100), moe(12, 4, 16, 0.5, (4, 2))),
        layer(latent(2, 16, 10, 40, 30, 130, 0.2, 10.0), moe(3, 1, 32, 1.0))]),
}
SEEDS = {"A": 41, "B": 42, "C": 43, "D": 44, "E": 45, "F": 46}
STD_SCALE = 0.8


def config(name: str):
    return telapel.config_from_json(RAW[name])


def write_raw_model(path: str, raw: dict, seed: int, std_scale: float = STD_SCALE,
                    edit: Optional[Callable[[Dict[str, torch.Tensor]], None]] = None) -> str:
    cfg = telapel.config_from_json(raw)
    tensors = random_tensors(cfg, seed, torch.bfloat16, std_scale)
    if edit is not None:
        edit(tensors)
    os.makedirs(path, exist_ok=True)
    write_config_json(path, cfg)
    save_file({k: v.contiguous() for k, v in tensors.items()}, os.path.join(path, "model.safetensors"))
    return path


def write_model(path: str, name: str, edit: Optional[Callable[[Dict[str, torch.Tensor]], None]] = None) -> str:
    return write_raw_model(path, RAW[name], SEEDS[name], edit=edit)


def random_raw(rng):
    """A random config.json: two to six layers of random types (some with an earlier layer's tensors), widths, head counts
    and sizes (also no multiples of 8), windows, taps, caps, temperatures, experts, groups, feed-forwards or none."""
    width = int(rng.choice([24, 40, 64, 72, 96, 136, 256]))

    def mixer():
        kind = rng.random()
        if kind < 0.34:
            blocks = int(rng.integers(1, 5))
            return rglru(blocks * int(rng.choice([6, 16, 20, 32, 48, 64, 80, 144, 272])), blocks, int(rng.choice([1, 2, 3, 4, 6, 9])))
        if kind < 0.67:
            return latent(int(rng.integers(1, 6)), int(rng.choice([4, 12, 16, 32, 50])), int(rng.choice([2, 6, 8, 16, 32])),
                          int(rng.choice([8, 16, 20, 64])), int(rng.choice([16, 20, 48, 72])), int(rng.choice([8, 20, 24, 48, 64, 96, 112, 150])),
                          float(rng.choice([0.1, 0.3])), float(rng.choice([10.0, 500.0, 1e4, 5e5])))
        kv = int(rng.integers(1, 4))
        return attention(kv * int(rng.integers(1, 4)), kv, int(rng.choice([8, 12, 16, 24, 32, 48, 64, 128])), float(rng.choice([0.1, 0.3])),
                         int(rng.choice([1, 2, 3, 4, 6])), float(rng.choice([0.0, 3.0, 20.0])),
                         int(rng.choice([0, 1, 2, 9, 16, 17, 50, 64, 70, 130, 300])),
                         (float(rng.choice([0.1, 0.7])), int(rng.choice([1, 5, 50, 1000]))) if rng.random() < 0.7 else None)

    def ff():
        if rng.random() < 0.25:
            return None
        count, size = int(rng.integers(1, 5)), int(rng.integers(1, 6))
        keep = int(rng.integers(1, count + 1))
        shared = int(rng.choice([0, 16, 36, 64]))
        return moe(count * size, int(rng.integers(1, min(keep * size, 4) + 1)), int(rng.choice([16, 24, 40, 100, 128])),
                   float(rng.choice([0.5, 1.0, 3.0])), (count, keep), (shared, float(rng.choice([0.4, 2.0]))) if shared else None)

    layers = []
    for i in range(int(rng.integers(2, 7))):
        if i and rng.random() < 0.25:
            j = int(rng.integers(0, i))
            layers.append(dict(layers[j], weights_of=j))
        else:
            layers.append(layer(mixer(), ff()))
    return model(int(rng.choice([50, 131, 300, 577])), width, float(rng.choice([1e-6, 1e-5])), layers)
