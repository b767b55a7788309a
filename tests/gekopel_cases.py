"""Small Gekopel configurations and model folders with random weights for the tests.

The configurations differ from each other in every size and option: the order of the layer types,
widths that are and are not multiples of 16, one head and several, one key/value head, a few and as
many as heads, query/key sizes below, at and above the value size, chunks of one position up to
longer than any request and none, bias tables of two to forty rows whose last bucket starts inside,
at and beyond a chunk, convolutions of one to five taps, dense and routed feed-forwards and none,
one to four experts a token out of two to twelve, one group, all groups kept and some left out,
groups of one expert, a shared expert or none."""

from __future__ import annotations

import dataclasses
import os
from typing import Callable, Dict, Optional

import torch
from safetensors.torch import save_file

from mini_gpt_inference_amd.config.model_config import write_config_json
from mini_gpt_inference_amd.models import gekopel
from mini_gpt_inference_amd.weights.random_init import random_tensors


def delta(heads, kv_heads, dim, vdim, conv):
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv}


def attention(heads, kv_heads, dim, vdim, scale, bias_max, chunk=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "bias_max": bias_max}
    if chunk:
        m["mask"] = {"size": chunk}
    return m


def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(experts, top, ff, groups=(1, 1), scale=1.0, shared=None):
    out = {"kind": "moe", "router": {"experts": experts, "top": top, "scale": scale,
                                     "groups": {"count": groups[0], "keep": groups[1]}}, "expert": {"ff": ff}}
    if shared:
        out["shared"] = {"ff": shared}
    return out


def layer(kind, mixer, mlp):
    return {"type": kind, "mixer": mixer, "mlp": mlp}


def model(vocab, width, eps, scale, max_positions, layers):
    return {"architecture": "Gekopel", "vocab": vocab, "width": width, "norm": {"eps": eps}, "embedding": {"scale": scale},
            "max_positions": max_positions, "layers": layers}


RAW: Dict[str, dict] = {
    # both mixers, all three kinds of feed-forward, a chunk shorter than a page and one longer than two, shared
    # queries and keys in the delta rule, groups of which one is left out
    "A": model(131, 64, 1e-5, 8.0, 500, [
        layer("attention", attention(4, 2, 16, 32, 0.25, 24, 7), dense(96)),
        layer("delta", delta(6, 2, 16, 24, 3), moe(6, 2, 48, (3, 2), 2.0, 40)),
        layer("attention", attention(2, 1, 24, 16, 0.2, 60, 37), moe(4, 1, 32, (2, 1), 0.7)),
        layer("delta", delta(3, 3, 8, 40, 2), None)]),
    # head sizes that the bfloat16 matrix-core attention kernels take (64 and 128), as many key/value heads as
    # heads, a delta layer first, no chunk, a last bucket within reach, groups of one expert, no shared expert
    "B": model(77, 96, 1e-6, 1.0, 300, [
        layer("delta", delta(2, 1, 64, 64, 5), moe(5, 2, 64, (5, 3), 1.0)),
        layer("attention", attention(2, 2, 64, 64, 0.125, 30), dense(80)),
        layer("attention", attention(1, 1, 128, 64, 0.09, 200, 50), moe(9, 3, 40, (3, 3), 1.25, 72))]),
    # a width and head sizes that only the general kernels take, chunks of one position (a token sees itself
    # only), one tap (no kept inputs), every expert chosen
    "C": model(59, 40, 1e-4, 3.5, 128, [
        layer("attention", attention(3, 1, 20, 12, 0.6, 9, 1), moe(2, 2, 24, (1, 1), 1.5, 24)),
        layer("delta", delta(4, 1, 12, 20, 1), dense(36)),
        layer("attention", attention(4, 2, 12, 20, 0.5, 41, 16), None),
        layer("delta", delta(2, 2, 36, 20, 4), moe(8, 3, 72, (2, 1), 0.5))]),
    # an attention layer, then a delta layer
    "D": model(33, 32, 1e-5, 2.0, 200, [
        layer("attention", attention(2, 1, 16, 16, 0.25, 50, 33), dense(64)),
        layer("delta", delta(2, 2, 16, 16, 4), moe(6, 2, 16, (2, 2), 1.0, 16))]),
    # delta layers only: no keys and values, no pages with anything in them
    "E": model(45, 48, 1e-5, 5.0, 150, [
        layer("delta", delta(4, 2, 24, 16, 4), moe(4, 2, 24, (4, 2), 1.0, 24)),
        layer("delta", delta(3, 1, 16, 32, 2), None)]),
    # attention layers only, two of them with the same pages and different chunks: no state
    "F": model(64, 80, 1e-5, 1.5, 260, [
        layer("attention", attention(4, 2, 32, 32, 0.18, 70, 40), moe(7, 1, 40, (7, 4), 1.0, 24)),
        layer("attention", attention(2, 2, 32, 24, 0.2, 7), None),
        layer("attention", attention(6, 2, 24, 32, 0.15, 300, 64), dense(112))]),
}
SEEDS = {"A": 31, "B": 32, "C": 33, "D": 34, "E": 35, "F": 36}
BUCKETS = {"A": 16, "B": 20, "C": 4, "D": 32, "E": 8, "F": 6}     # rows of the distance tables
STD_SCALE = 1.5


def with_buckets(cfg, buckets: int):
    """config.json does not say how many rows a distance table has (the stored tensors do): random weights are drawn
    with the number given here."""
    layers = tuple(dataclasses.replace(l, mixer=dataclasses.replace(l.mixer, buckets=buckets)) if l.type == "attention" else l
                   for l in cfg.layers)
    return dataclasses.replace(cfg, layers=layers)


def config(name: str):
    return with_buckets(gekopel.config_from_json(RAW[name]), BUCKETS[name])


def write_raw_model(path: str, raw: dict, seed: int, std_scale: float = STD_SCALE, buckets: int = 32,
                    edit: Optional[Callable[[Dict[str, torch.Tensor]], None]] = None) -> str:
    cfg = with_buckets(gekopel.config_from_json(raw), buckets)
    tensors = random_tensors(cfg, seed, torch.bfloat16, std_scale)
    if edit is not None:
        edit(tensors)
    os.makedirs(path, exist_ok=True)
    write_config_json(path, cfg)
    save_file({k: v.contiguous() for k, v in tensors.items()}, os.path.join(path, "model.safetensors"))
    return path


def write_model(path: str, name: str, edit: Optional[Callable[[Dict[str, torch.Tensor]], None]] = None) -> str:
    return write_raw_model(path, RAW[name], SEEDS[name], buckets=BUCKETS[name], edit=edit)


def random_raw(rng):
    """A random config.json and a number of distance buckets that suits it: two to six layers of random types, widths,
    head counts and sizes (also no multiples of 8), chunks, taps, experts, groups, feed-forwards or none."""
    width = int(rng.choice([24, 40, 64, 72, 96, 136, 256]))
    buckets = int(rng.choice([2, 4, 6, 16, 32, 40]))

    def att():
        dim, vdim = int(rng.choice([8, 12, 16, 24, 32, 48, 64, 128])), int(rng.choice([8, 16, 20, 32, 64, 128]))
        kv = int(rng.integers(1, 4))
        return attention(kv * int(rng.integers(1, 4)), kv, dim, vdim, float(rng.choice([0.1, 0.3, dim ** -0.5])),
                         buckets // 2 + int(rng.choice([1, 2, 7, 30, 100, 400])),
                         int(rng.choice([0, 1, 2, 9, 16, 17, 50, 64, 70, 130, 300])))

    def ff():
        kind = rng.random()
        if kind < 0.2:
            return None
        hidden = int(rng.choice([16, 24, 40, 100, 128]))
        if kind < 0.45:
            return dense(hidden)
        count, size = int(rng.integers(1, 5)), int(rng.integers(1, 6))
        keep = int(rng.integers(1, count + 1))
        return moe(count * size, int(rng.integers(1, min(keep * size, 4) + 1)), hidden, (count, keep),
                   float(rng.choice([0.5, 1.0, 2.5])), int(rng.choice([0, 16, 36, 64])) or None)

    layers = []
    for _ in range(int(rng.integers(2, 7))):
        if rng.random() < 0.5:
            kv = int(rng.integers(1, 4))
            layers.append(layer("delta", delta(kv * int(rng.integers(1, 4)), kv, int(rng.choice([8, 12, 16, 32, 48, 64, 128, 136])),
                                               int(rng.choice([8, 16, 20, 32, 64, 128])), int(rng.choice([1, 2, 3, 4, 6]))), ff()))
        else:
            layers.append(layer("attention", att(), ff()))
    return model(int(rng.choice([50, 131, 300, 577])), width, float(rng.choice([1e-6, 1e-5])),
                 float(rng.choice([1.0, 6.0, width ** 0.5])), int(rng.choice([200, 256, 333])), layers), buckets
