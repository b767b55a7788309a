"""Gekopel: a decoder whose layers are listed one by one in config.json, each with the gated delta rule or a
chunked softmax attention as its mixer, dense or routed feed-forwards, and learned positions, as data.

What the design fixes, and is therefore set here and handed to the parts as parameters:
- the embedded tokens are multiplied by `embedding.scale`; a learned row per position (`pos`, not scaled) is added;
- every norm is an RMS norm with a plain gain and one eps (config `norm.eps`); a layer norms each sublayer on both
  sides (the `sandwich_norm` arrangement); `mlp: null` leaves the feed-forward out;
- layer type `delta`: the gated delta rule; `heads` value heads of size `vdim`, `kv_heads` query/key heads of size
  `dim`, a short convolution of `conv` taps with silu behind each of the three projections, unit queries (times
  dim^-1/2) and keys, one decay and one step size per head, each head's output normed with one weight that the
  heads share, a silu gate;
- layer type `attention`: grouped softmax attention without biases and without rotation; scores times `scale` plus
  a learned number per head and distance bucket (`rel`, buckets up to `bias_max`), a sink per head in the softmax's
  denominator, chunks of `mask.size` positions;
- feed-forward `dense`: down(relu(up h)^2);
- feed-forward `moe`: `router.experts` experts of the same form and hidden size `expert.ff`; sigmoid scores, chosen
  by score plus correction among the `router.groups.keep` best of `router.groups.count` groups, weights the
  scores divided by their sum times `router.scale`, on the experts' outputs; a shared expert of hidden size
  `shared.ff` times a sigmoid number per token;
- the head: the model's norm (`final.norm`), then `head`, untied.

Tensor names: `embed`, `pos`, `l<i>.norm1|norm1b|norm2|norm2b`, `l<i>.mix.{q,k,v,q.conv,k.conv,v.conv,b,a,A_log,
dt_bias,norm,g,o}` (delta), `l<i>.mix.{q,k,v,rel,sink,o}` (attention), `l<i>.mlp.{up,down}` (dense),
`l<i>.mlp.{router,correction}`, `l<i>.mlp.e<j>.{up,down}`, `l<i>.mlp.shared.{up,down,sg}` (moe), `final.norm`,
`head`; linear weights are stored [out, in].
"""

from __future__ import annotations

import math
from dataclasses import dataclass
from typing import Any, Dict, List, Mapping, Optional, Tuple

from ..config.model_config import ConfigError
from ..config.registry import Architecture, register_architecture
from ..parts.base import PartSpec
from ..parts.model import LayerRun, LayerSpec, ModelSpec

NAME = "Gekopel"


@dataclass(frozen=True)
class DeltaConfig:
    heads: int
    kv_heads: int               # query/key heads, shared by heads / kv_heads value heads each
    dim: int
    vdim: int
    conv: int                   # taps of the short convolutions


@dataclass(frozen=True)
class ChunkAttentionConfig:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    bias_max: int               # distance from which on all keys share the last bucket
    chunk: int = 0              # positions of a chunk, counted from position 0; 0: all earlier keys are seen
    # rows of the distance table.  config.json does not carry them: a model folder's tensors give them by their
    # shape; this value is what random weights are drawn with
    buckets: int = 32


@dataclass(frozen=True)
class DenseConfig:
    ff: int


@dataclass(frozen=True)
class ExpertsConfig:
    experts: int
    top: int
    ff: int
    scale: float = 1.0
    groups: int = 1
    keep: int = 1
    shared_ff: int = 0          # hidden size of the shared expert, 0: none


@dataclass(frozen=True)
class LayerConfig:
    type: str                                   # "delta" or "attention"
    mixer: Any                                  # DeltaConfig or ChunkAttentionConfig
    mlp: Any                                    # DenseConfig, ExpertsConfig or None: no feed-forward


@dataclass(frozen=True)
class GekopelConfig:
    architecture: str
    vocab: int
    width: int
    max_positions: int
    layers: Tuple[LayerConfig, ...]
    norm_eps: float
    embedding_scale: float = 1.0


def _positive(name: str, value: Any) -> int:
    if not isinstance(value, int) or isinstance(value, bool) or value <= 0:
        raise ConfigError(f"{name} must be a positive integer, got {value!r}")
    return value


def _heads(where: str, m: Mapping[str, Any]) -> Tuple[int, int, int, int]:
    heads, kv_heads = _positive(f"{where} heads", m.get("heads")), _positive(f"{where} kv_heads", m.get("kv_heads"))
    if heads % kv_heads:
        raise ConfigError(f"{where}: heads must be a multiple of kv_heads")
    return heads, kv_heads, _positive(f"{where} dim", m.get("dim")), _positive(f"{where} vdim", m.get("vdim"))


def _attention(where: str, m: Mapping[str, Any]) -> ChunkAttentionConfig:
    chunk = (m.get("mask") or {}).get("size") or 0
    if not isinstance(chunk, int) or chunk < 0:
        raise ConfigError(f"{where}: mask.size must be a non-negative integer")
    return ChunkAttentionConfig(*_heads(where, m), float(m["scale"]), _positive(f"{where} bias_max", m.get("bias_max")), chunk)


def _mlp(where: str, mlp: Optional[Mapping[str, Any]]) -> Any:
    if mlp is None:
        return None
    kind = mlp.get("kind")
    if kind == "dense":
        return DenseConfig(_positive(f"{where} ff", mlp.get("ff")))
    if kind != "moe":
        raise ConfigError(f"{where}: unknown feed-forward kind {kind!r}")
    router, expert, shared = mlp.get("router") or {}, mlp.get("expert") or {}, mlp.get("shared") or {}
    n, top = _positive(f"{where} router.experts", router.get("experts")), _positive(f"{where} router.top", router.get("top"))
    groups = router.get("groups") or {"count": 1, "keep": 1}
    count, keep = _positive(f"{where} groups.count", groups.get("count")), _positive(f"{where} groups.keep", groups.get("keep"))
    if keep > count or n % count or top > keep * (n // count):
        raise ConfigError(f"{where}: top {top} of {n} experts in {count} groups of which {keep} stay")
    return ExpertsConfig(n, top, _positive(f"{where} expert.ff", expert.get("ff")), float(router.get("scale", 1.0)), count, keep,
                         _positive(f"{where} shared.ff", shared.get("ff")) if shared else 0)


def config_from_json(raw: Mapping[str, Any]) -> GekopelConfig:
    if not isinstance(raw.get("layers"), list) or not raw["layers"]:
        raise ConfigError("config.json lists no layers")
    layers: List[LayerConfig] = []
    for i, layer in enumerate(raw["layers"]):
        kind, m = layer.get("type"), layer.get("mixer")
        if not isinstance(m, Mapping):
            raise ConfigError(f"layer {i}: no mixer sizes")
        if kind == "delta":
            mixer: Any = DeltaConfig(*_heads(f"layer {i}", m), _positive(f"layer {i} conv", m.get("conv")))
        elif kind == "attention":
            mixer = _attention(f"layer {i}", m)
        else:
            raise ConfigError(f"layer {i}: unknown mixer type {kind!r}")
        layers.append(LayerConfig(kind, mixer, _mlp(f"layer {i} mlp", layer.get("mlp"))))
    return GekopelConfig(architecture=NAME, vocab=_positive("vocab", raw.get("vocab")),
                         width=_positive("width", raw.get("width")),
                         max_positions=_positive("max_positions", raw.get("max_positions")), layers=tuple(layers),
                         norm_eps=float(raw["norm"]["eps"]),
                         embedding_scale=float((raw.get("embedding") or {}).get("scale", 1.0)))


def config_to_json(cfg: GekopelConfig) -> Dict[str, Any]:
    layers = []
    for layer in cfg.layers:
        m = layer.mixer
        mixer: Dict[str, Any] = {"heads": m.heads, "kv_heads": m.kv_heads, "dim": m.dim, "vdim": m.vdim}
        if layer.type == "delta":
            mixer["conv"] = m.conv
        else:
            mixer.update(scale=m.scale, bias_max=m.bias_max)
            if m.chunk:
                mixer["mask"] = {"size": m.chunk}
        f = layer.mlp
        if isinstance(f, DenseConfig):
            mlp: Optional[Dict[str, Any]] = {"kind": "dense", "ff": f.ff}
        elif f is not None:
            mlp = {"kind": "moe", "expert": {"ff": f.ff},
                   "router": {"experts": f.experts, "top": f.top, "scale": f.scale,
                              "groups": {"count": f.groups, "keep": f.keep}}}
            if f.shared_ff:
                mlp["shared"] = {"ff": f.shared_ff}
        else:
            mlp = None
        layers.append({"type": layer.type, "mixer": mixer, "mlp": mlp})
    return {"architecture": NAME, "vocab": cfg.vocab, "width": cfg.width, "max_positions": cfg.max_positions,
            "embedding": {"scale": cfg.embedding_scale}, "norm": {"eps": cfg.norm_eps}, "layers": layers}


def model_spec(cfg: GekopelConfig) -> ModelSpec:
    w, eps = cfg.width, cfg.norm_eps

    def norm(name: str) -> PartSpec:
        return PartSpec("rms_norm", {"width": w, "eps": eps, "one_plus": False}, {"weight": name})

    def delta(m: DeltaConfig, p: str) -> PartSpec:
        return PartSpec(
            "gated_delta_rule",
            {"width": w, "n_head": m.heads, "n_kv_head": m.kv_heads, "head_dim": m.dim, "value_dim": m.vdim,
             "conv_taps": m.conv, "norm_eps": eps, "q_scale": m.dim ** -0.5},
            {"q_weight": p + "q", "k_weight": p + "k", "v_weight": p + "v", "gate_weight": p + "g", "beta_weight": p + "b",
             "decay_weight": p + "a", "q_conv": p + "q.conv", "k_conv": p + "k.conv", "v_conv": p + "v.conv",
             "a_log": p + "A_log", "dt_bias": p + "dt_bias", "norm_weight": p + "norm", "out_weight": p + "o"})

    def attention(m: ChunkAttentionConfig, p: str) -> PartSpec:
        return PartSpec(
            "gated_attention",
            {"width": w, "n_head": m.heads, "n_kv_head": m.kv_heads, "head_dim": m.dim, "value_dim": m.vdim,
             "scale": m.scale, "sinks": True, "window": m.chunk, "chunked": True, "bias_max": m.bias_max},
            {"q_weight": p + "q", "k_weight": p + "k", "v_weight": p + "v", "out_weight": p + "o", "sink": p + "sink",
             "rel": p + "rel"})

    def feed_forward(f: Any, p: str) -> PartSpec:
        if isinstance(f, DenseConfig):
            return PartSpec("dense_mlp", {"width": w, "hidden": f.ff, "bias": False, "activation": "relu2"},
                            {"fc_weight": p + "up", "proj_weight": p + "down"})
        names = {"router_weight": p + "router", "correction": p + "correction"}
        for e in range(f.experts):
            names.update({f"e{e}_up": f"{p}e{e}.up", f"e{e}_down": f"{p}e{e}.down"})
        if f.shared_ff:
            names.update(shared_up=p + "shared.up", shared_down=p + "shared.down", shared_gate_weight=p + "shared.sg")
        return PartSpec(
            "routed_experts",
            {"width": w, "hidden": f.ff, "n_experts": f.experts, "top": f.top, "shared_hidden": f.shared_ff,
             "score": "sigmoid", "activation": "relu2", "weight_on": "output", "correction": True,
             "groups": (f.groups, f.keep), "normalise": True, "scale": f.scale, "shared_gate": True}, names)

    layers = []
    for i, layer in enumerate(cfg.layers):
        p = f"l{i}."
        mixer = delta(layer.mixer, p + "mix.") if layer.type == "delta" else attention(layer.mixer, p + "mix.")
        parts: Dict[str, Tuple[str, PartSpec]] = {"norm1": ("norm", norm(p + "norm1")), "mixer": ("mixer", mixer),
                                                  "norm1b": ("norm", norm(p + "norm1b"))}
        if layer.mlp is not None:
            parts["norm2"] = ("norm", norm(p + "norm2"))
            parts["feed_forward"] = ("feed_forward", feed_forward(layer.mlp, p + "mlp."))
            parts["norm2b"] = ("norm", norm(p + "norm2b"))
        arrangement = PartSpec("sandwich_norm", {"width": w, "feed_forward": layer.mlp is not None})
        layers.append(LayerSpec(arrangement, parts=parts))
    return ModelSpec(
        width=w, vocab_size=cfg.vocab,
        embedding=PartSpec("token_embedding", {"vocab_size": cfg.vocab, "width": w, "scale": cfg.embedding_scale},
                           {"weight": "embed"}),
        position=PartSpec("learned_absolute", {"max_positions": cfg.max_positions, "width": w}, {"weight": "pos"}),
        layers=tuple(layers), order=tuple(LayerRun(i) for i in range(len(layers))),
        final_norm=norm("final.norm"),
        head=PartSpec("linear_head", {"vocab_size": cfg.vocab, "width": w, "tied": False}, {"weight": "head"}),
        max_positions=cfg.max_positions)


def init_plan(cfg: GekopelConfig) -> List[Tuple[str, Tuple[int, ...], str, float]]:
    """Random-weights rule, in drawing order: matrices N(0, 1/sqrt(fan_in)), the embedding so that the scaled rows are
    N(0, 1), positions and distance numbers N(0, 0.5), convolution taps N(0, 1/sqrt(taps)), gains 1 + N(0, 0.1), decay
    constants around values between fast and slow, corrections N(0, 0.1), sinks N(0, 1)."""
    w = cfg.width
    plan: List[Tuple[str, Tuple[int, ...], str, float]] = [
        ("embed", (cfg.vocab, w), "normal", 1.0 / max(abs(cfg.embedding_scale), 1e-6)),
        ("pos", (cfg.max_positions, w), "normal", 0.5)]

    def lin(name: str, out: int, inn: int) -> None:
        plan.append((name, (out, inn), "normal", 1.0 / math.sqrt(inn)))

    for i, layer in enumerate(cfg.layers):
        p, m, f = f"l{i}.", layer.mixer, layer.mlp
        q = p + "mix."
        for n in ("norm1", "norm1b") + (("norm2", "norm2b") if f is not None else ()):
            plan.append((p + n, (w,), "gain", 0.1))
        for n, out in (("q", (m.kv_heads if layer.type == "delta" else m.heads) * m.dim), ("k", m.kv_heads * m.dim),
                       ("v", (m.heads if layer.type == "delta" else m.kv_heads) * m.vdim)):
            lin(q + n, out, w)
            if layer.type == "delta":
                plan.append((q + n + ".conv", (out, m.conv), "normal", 1.0 / math.sqrt(m.conv)))
        if layer.type == "delta":
            lin(q + "b", m.heads, w)
            lin(q + "a", m.heads, w)
            plan.append((q + "A_log", (m.heads,), "around", 0.0))
            plan.append((q + "dt_bias", (m.heads,), "around", -2.0))
            plan.append((q + "norm", (m.vdim,), "gain", 0.1))
            lin(q + "g", m.heads * m.vdim, w)
        else:
            plan.append((q + "rel", (m.buckets, m.heads), "normal", 0.5))
            plan.append((q + "sink", (m.heads,), "normal", 1.0))
        lin(q + "o", w, m.heads * m.vdim)
        if isinstance(f, DenseConfig):
            lin(p + "mlp.up", f.ff, w)
            lin(p + "mlp.down", w, f.ff)
        elif f is not None:
            for e in range(f.experts):
                lin(f"{p}mlp.e{e}.up", f.ff, w)
                lin(f"{p}mlp.e{e}.down", w, f.ff)
            lin(p + "mlp.router", f.experts, w)
            plan.append((p + "mlp.correction", (f.experts,), "normal", 0.1))
            if f.shared_ff:
                lin(p + "mlp.shared.up", f.shared_ff, w)
                lin(p + "mlp.shared.down", w, f.shared_ff)
                lin(p + "mlp.shared.sg", 1, w)
    plan.append(("final.norm", (w,), "gain", 0.1))
    lin("head", cfg.vocab, w)
    return plan


register_architecture(Architecture(NAME, config_from_json, model_spec, init_plan, config_to_json))
