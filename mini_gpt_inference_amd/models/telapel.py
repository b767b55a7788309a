"""Telapel: a decoder whose layers are listed one by one in config.json, each with a gated diagonal recurrence, latent
attention or windowed attention as its mixer and routed experts as its feed-forward, as data.

What the design fixes, and is therefore set here and handed to the parts as parameters:
- no position table; the head is the embedding table;
- every norm is an RMS norm with a plain gain and one eps (config `norm.eps`); a layer norms each sublayer's output only
  (the `sandwich_norm` arrangement without input norms): the sublayers read the residual itself; `mlp: null` leaves the
  feed-forward out;
- layer type `rglru`: a gelu branch and a convolved branch of `width` channels, one number of state per channel whose
  decay and input gate come from `blocks` square matrices each, log decay -8 r softplus(lam);
- layer type `latent_attention`: queries from a normed latent of `q_rank` values; keys and values made from a cached
  latent of `kv_rank` values beside one rotated key part of `rot_dim` channels that all heads share; a query head is
  [dim plain | rot_dim rotated]; neighbouring channels are rotated as pairs; causal softmax, no gate, no sink;
- layer type `attention`: grouped heads with biases on queries and keys, which pass a short convolution of `conv` taps and
  an RMS norm per head with one weight vector; the values are the keys as they leave the convolution; no rotation; queries
  times a temperature that grows with the position (`q_temp`), scores capped (`softcap`), then a slope per head
  times the distance taken off; a window of `mask.size` positions; a sink of score 0;
- feed-forward `moe`: `router.experts` experts with the clamped swish unit (sharpness 1.702, `expert.limit`), softmax
  scores, the `router.top` best of the `router.groups.keep` groups (of `router.groups.count`) with the best experts,
  weights the chosen scores divided by their sum, on the experts' outputs; beside them a shared one (`shared.ff`, `shared.limit`);
- a layer with `weights_of: j` runs layer j's parts once more; its cache or state is separate.

Tensor names: `embed`, `l<i>.norm1|norm2`, `l<i>.mix.{y,y.b,x,x.b,conv,conv.b,ra,ra.b,ri,ri.b,lam,o}` (rglru),
`l<i>.mix.{dq,dq.norm,uq,dkv,dkv.norm,uk,uv,o}` (latent_attention), `l<i>.mix.{q,k,q.b,k.b,q.conv,k.conv,q.norm,k.norm,o}`
(attention), `l<i>.mlp.router`, `l<i>.mlp.e<j>.{gate,up,down}`, `l<i>.mlp.shared.{gate,up,down}`, `final.norm`; matrices
are [out, in].
"""

from __future__ import annotations

import math
from dataclasses import dataclass
from typing import Any, Dict, List, Mapping, Optional, Tuple

from ..config.model_config import ConfigError
from ..config.registry import Architecture, register_architecture
from ..parts.base import PartSpec
from ..parts.mixers import geometric_slopes
from ..parts.model import LayerRun, LayerSpec, ModelSpec

NAME = "Telapel"
DECAY_SCALE = 8.0           # log decay = -8 r softplus(lam)
SWISH_SHARPNESS = 1.702     # of the experts' unit
SINK_SCORE = 0.0            # the windowed attention's sink


@dataclass(frozen=True)
class RecurrentConfig:
    channels: int               # the config's mixer.width
    blocks: int
    conv: int                   # taps of the short convolution


@dataclass(frozen=True)
class LatentConfig:
    heads: int
    dim: int
    rot_dim: int
    vdim: int
    q_rank: int
    kv_rank: int
    scale: float
    rot_base: float


@dataclass(frozen=True)
class WindowConfig:
    heads: int
    kv_heads: int
    dim: int                    # of queries, keys and values
    scale: float
    conv: int
    softcap: float = 0.0        # 0: scores are not capped
    window: int = 0             # positions a query sees, its own included; 0: all
    temp_coef: float = 0.0
    temp_every: int = 0         # 0: no query temperature


@dataclass(frozen=True)
class ExpertsConfig:
    experts: int
    top: int
    ff: int
    limit: float
    groups: int = 1
    keep: int = 1
    shared_ff: int = 0          # hidden size of the shared expert, 0: none
    shared_limit: float = 0.0


@dataclass(frozen=True)
class LayerConfig:
    type: str                               # "rglru", "latent_attention" or "attention"
    mixer: Any
    mlp: Optional[ExpertsConfig]            # None: no feed-forward
    weights_of: Optional[int] = None        # the layer whose tensors this one uses; None: its own


@dataclass(frozen=True)
class TelapelConfig:
    architecture: str
    vocab: int
    width: int
    layers: Tuple[LayerConfig, ...]
    norm_eps: float


def _positive(name: str, value: Any) -> int:
    if not isinstance(value, int) or isinstance(value, bool) or value <= 0:
        raise ConfigError(f"{name} must be a positive integer, got {value!r}")
    return value


def _recurrent(where: str, m: Mapping[str, Any]) -> RecurrentConfig:
    channels, blocks = _positive(f"{where} width", m.get("width")), _positive(f"{where} blocks", m.get("blocks"))
    if channels % blocks:
        raise ConfigError(f"{where}: width must be a multiple of blocks")
    return RecurrentConfig(channels, blocks, _positive(f"{where} conv", m.get("conv")))


def _latent(where: str, m: Mapping[str, Any]) -> LatentConfig:
    rot_dim, rot = _positive(f"{where} rot_dim", m.get("rot_dim")), m.get("rot")
    if not isinstance(rot, Mapping) or rot.get("dims", rot_dim) != rot_dim or rot_dim % 2:
        raise ConfigError(f"{where}: the rotation covers the rotated part, rot.dims = rot_dim, an even number")
    if not float(rot.get("base", 0.0)) > 0.0:
        raise ConfigError(f"{where}: rot.base must be positive")
    return LatentConfig(_positive(f"{where} heads", m.get("heads")), _positive(f"{where} dim", m.get("dim")), rot_dim,
                        _positive(f"{where} vdim", m.get("vdim")), _positive(f"{where} q_rank", m.get("q_rank")),
                        _positive(f"{where} kv_rank", m.get("kv_rank")), float(m["scale"]), float(rot["base"]))


def _window(where: str, m: Mapping[str, Any]) -> WindowConfig:
    heads, kv_heads = _positive(f"{where} heads", m.get("heads")), _positive(f"{where} kv_heads", m.get("kv_heads"))
    dim = _positive(f"{where} dim", m.get("dim"))
    if heads % kv_heads:
        raise ConfigError(f"{where}: heads must be a multiple of kv_heads")
    if m.get("vdim", dim) != dim:
        raise ConfigError(f"{where}: the values are the keys, so vdim = dim")
    window = (m.get("mask") or {}).get("size") or 0
    softcap = float(m.get("softcap") or 0.0)
    if not isinstance(window, int) or window < 0 or softcap < 0.0:
        raise ConfigError(f"{where}: mask.size must be a non-negative integer, softcap not negative")
    temp = m.get("q_temp") or {}
    every = 0
    if temp:
        every = temp.get("every")
        every = _positive(f"{where} q_temp.every", int(every) if isinstance(every, float) and every.is_integer() else every)
    return WindowConfig(heads, kv_heads, dim, float(m["scale"]), _positive(f"{where} conv", m.get("conv")), softcap, window,
                        float(temp.get("coef", 0.0)), every)


def _limit(where: str, m: Mapping[str, Any]) -> float:
    limit = float(m["limit"])
    if not limit > 0.0:
        raise ConfigError(f"{where}: limit must be positive")
    return limit


def _experts(where: str, mlp: Optional[Mapping[str, Any]]) -> Optional[ExpertsConfig]:
    if mlp is None:
        return None
    if mlp.get("kind") != "moe":
        raise ConfigError(f"{where}: unknown feed-forward kind {mlp.get('kind')!r}")
    router, expert, shared = mlp.get("router") or {}, mlp.get("expert") or {}, mlp.get("shared") or {}
    n, top = _positive(f"{where} router.experts", router.get("experts")), _positive(f"{where} router.top", router.get("top"))
    groups = router.get("groups") or {"count": 1, "keep": 1}
    count, keep = _positive(f"{where} groups.count", groups.get("count")), _positive(f"{where} groups.keep", groups.get("keep"))
    if keep > count or n % count or top > keep * (n // count):
        raise ConfigError(f"{where}: top {top} of {n} experts in {count} groups of which {keep} stay")
    return ExpertsConfig(n, top, _positive(f"{where} expert.ff", expert.get("ff")), _limit(f"{where} expert", expert), count, keep,
                         _positive(f"{where} shared.ff", shared.get("ff")) if shared else 0,
                         _limit(f"{where} shared", shared) if shared else 0.0)


_MIXERS = {"rglru": _recurrent, "latent_attention": _latent, "attention": _window}


def config_from_json(raw: Mapping[str, Any]) -> TelapelConfig:
    if not isinstance(raw.get("layers"), list) or not raw["layers"]:
        raise ConfigError("config.json lists no layers")
    layers: List[LayerConfig] = []
    for i, layer in enumerate(raw["layers"]):
        kind, m = layer.get("type"), layer.get("mixer")
        if kind not in _MIXERS:
            raise ConfigError(f"layer {i}: unknown mixer type {kind!r}")
        if not isinstance(m, Mapping):
            raise ConfigError(f"layer {i}: no mixer sizes")
        made = LayerConfig(kind, _MIXERS[kind](f"layer {i}", m), _experts(f"layer {i} mlp", layer.get("mlp")), layer.get("weights_of"))
        j = made.weights_of
        if j is not None:
            if not isinstance(j, int) or isinstance(j, bool) or not 0 <= j < i:
                raise ConfigError(f"layer {i}: weights_of names an earlier layer")
            if (layers[j].type, layers[j].mixer, layers[j].mlp) != (made.type, made.mixer, made.mlp):
                raise ConfigError(f"layer {i}: differs from layer {j}, whose tensors it uses")
        layers.append(made)
    return TelapelConfig(architecture=NAME, vocab=_positive("vocab", raw.get("vocab")), width=_positive("width", raw.get("width")),
                         layers=tuple(layers), norm_eps=float(raw["norm"]["eps"]))


def config_to_json(cfg: TelapelConfig) -> Dict[str, Any]:
    layers = []
    for layer in cfg.layers:
        m, f = layer.mixer, layer.mlp
        if layer.type == "rglru":
            mixer: Dict[str, Any] = {"width": m.channels, "blocks": m.blocks, "conv": m.conv}
        elif layer.type == "latent_attention":
            mixer = {"heads": m.heads, "dim": m.dim, "rot_dim": m.rot_dim, "vdim": m.vdim, "q_rank": m.q_rank,
                     "kv_rank": m.kv_rank, "scale": m.scale, "rot": {"base": m.rot_base, "dims": m.rot_dim}}
        else:
            mixer = {"heads": m.heads, "kv_heads": m.kv_heads, "dim": m.dim, "vdim": m.dim, "scale": m.scale, "conv": m.conv}
            if m.softcap:
                mixer["softcap"] = m.softcap
            if m.window:
                mixer["mask"] = {"size": m.window}
            if m.temp_every:
                mixer["q_temp"] = {"coef": m.temp_coef, "every": m.temp_every}
        mlp: Optional[Dict[str, Any]] = None
        if f is not None:
            mlp = {"kind": "moe", "expert": {"ff": f.ff, "limit": f.limit},
                   "router": {"experts": f.experts, "top": f.top, "groups": {"count": f.groups, "keep": f.keep}}}
            if f.shared_ff:
                mlp["shared"] = {"ff": f.shared_ff, "limit": f.shared_limit}
        entry = {"type": layer.type, "mixer": mixer, "mlp": mlp}
        if layer.weights_of is not None:
            entry["weights_of"] = layer.weights_of
        layers.append(entry)
    return {"architecture": NAME, "vocab": cfg.vocab, "width": cfg.width, "norm": {"eps": cfg.norm_eps}, "layers": layers}


def _owner(cfg: TelapelConfig, i: int) -> int:
    """The layer whose tensors layer i uses, itself mostly."""
    while cfg.layers[i].weights_of is not None:
        i = cfg.layers[i].weights_of
    return i


def model_spec(cfg: TelapelConfig) -> ModelSpec:
    w, eps = cfg.width, cfg.norm_eps

    def norm(name: str) -> PartSpec:
        return PartSpec("rms_norm", {"width": w, "eps": eps, "one_plus": False}, {"weight": name})

    def recurrent(m: RecurrentConfig, p: str) -> PartSpec:
        return PartSpec(
            "gated_diagonal_state",
            {"width": w, "channels": m.channels, "blocks": m.blocks, "conv_taps": m.conv, "decay_scale": DECAY_SCALE},
            {"y_weight": p + "y", "y_bias": p + "y.b", "x_weight": p + "x", "x_bias": p + "x.b", "conv_weight": p + "conv",
             "conv_bias": p + "conv.b", "r_weight": p + "ra", "r_bias": p + "ra.b", "i_weight": p + "ri", "i_bias": p + "ri.b",
             "lam": p + "lam", "out_weight": p + "o"})

    def latent(m: LatentConfig, p: str) -> PartSpec:
        return PartSpec(
            "latent_attention",
            {"width": w, "n_head": m.heads, "head_dim": m.dim, "value_dim": m.vdim, "rank": m.kv_rank, "scale": m.scale,
             "eps": eps, "rot_dim": m.rot_dim, "rotary": {"kind": "rotary_interleaved", "dims": m.rot_dim, "base": m.rot_base},
             "gate": None, "sinks": False, "q_rank": m.q_rank},
            {"dq_weight": p + "dq", "dq_norm": p + "dq.norm", "q_weight": p + "uq", "dkv_weight": p + "dkv",
             "dkv_norm": p + "dkv.norm", "uk_weight": p + "uk", "uv_weight": p + "uv", "out_weight": p + "o"})

    def window(m: WindowConfig, p: str) -> PartSpec:
        return PartSpec(
            "gated_attention",
            {"width": w, "n_head": m.heads, "n_kv_head": m.kv_heads, "head_dim": m.dim, "value_dim": m.dim, "scale": m.scale,
             "bias": True, "conv_taps": m.conv, "values_from_keys": True, "qk_norm_eps": eps, "qk_norm_weights": "head",
             "query_temperature": (m.temp_coef, m.temp_every) if m.temp_every else None, "softcap": m.softcap,
             "slopes": geometric_slopes(m.heads), "window": m.window, "sink_score": SINK_SCORE},
            {"q_weight": p + "q", "k_weight": p + "k", "q_bias": p + "q.b", "k_bias": p + "k.b", "q_conv": p + "q.conv",
             "k_conv": p + "k.conv", "q_norm": p + "q.norm", "k_norm": p + "k.norm", "out_weight": p + "o"})

    def experts(f: ExpertsConfig, p: str) -> PartSpec:
        names = {"router_weight": p + "router"}
        for e in range(f.experts):
            names.update({f"e{e}_gate": f"{p}e{e}.gate", f"e{e}_up": f"{p}e{e}.up", f"e{e}_down": f"{p}e{e}.down"})
        if f.shared_ff:
            names.update(shared_gate=p + "shared.gate", shared_up=p + "shared.up", shared_down=p + "shared.down")
        return PartSpec(
            "routed_experts",
            {"width": w, "hidden": f.ff, "n_experts": f.experts, "top": f.top, "shared_hidden": f.shared_ff, "score": "softmax",
             "activation": "clamped_swish", "limit": f.limit, "shared_limit": f.shared_limit or None,
             "sharpness": SWISH_SHARPNESS, "weight_on": "output", "groups": (f.groups, f.keep), "group_best": 1,
             "normalise": True}, names)

    mixers = {"rglru": recurrent, "latent_attention": latent, "attention": window}
    layers: List[LayerSpec] = []
    place: Dict[int, int] = {}      # config layer -> its place among the distinct layers
    order: List[LayerRun] = []
    for i, layer in enumerate(cfg.layers):
        if _owner(cfg, i) == i:
            p = f"l{i}."
            parts: Dict[str, Tuple[str, PartSpec]] = {"mixer": ("mixer", mixers[layer.type](layer.mixer, p + "mix.")),
                                                      "norm1b": ("norm", norm(p + "norm1"))}
            if layer.mlp is not None:
                parts["feed_forward"] = ("feed_forward", experts(layer.mlp, p + "mlp."))
                parts["norm2b"] = ("norm", norm(p + "norm2"))
            place[i] = len(layers)
            layers.append(LayerSpec(PartSpec("sandwich_norm", {"width": w, "feed_forward": layer.mlp is not None, "input_norm": False}),
                                    parts=parts))
        order.append(LayerRun(place[_owner(cfg, i)]))
    return ModelSpec(
        width=w, vocab_size=cfg.vocab,
        embedding=PartSpec("token_embedding", {"vocab_size": cfg.vocab, "width": w}, {"weight": "embed"}),
        position=PartSpec("none"),
        layers=tuple(layers), order=tuple(order),
        final_norm=norm("final.norm"),
        head=PartSpec("linear_head", {"vocab_size": cfg.vocab, "width": w, "tied": True}, {"weight": "embed"}),
        max_positions=None)


def init_plan(cfg: TelapelConfig) -> List[Tuple[str, Tuple[int, ...], str, float]]:
    """Random-weights rule, in drawing order: matrices N(0, 1/sqrt(fan_in)), the embedding N(0, 1), biases N(0, 0.3),
    convolution taps N(0, 1/sqrt(taps)), gains 1 + N(0, 0.1), lam around a value that gives decays between fast and slow."""
    w = cfg.width
    plan: List[Tuple[str, Tuple[int, ...], str, float]] = [("embed", (cfg.vocab, w), "normal", 1.0)]

    def lin(name: str, out: int, inn: int, bias: bool = False) -> None:
        plan.append((name, (out, inn), "normal", 1.0 / math.sqrt(inn)))
        if bias:
            plan.append((name + ".b", (out,), "normal", 0.3))

    for i, layer in enumerate(cfg.layers):
        if layer.weights_of is not None:
            continue
        p, m, f = f"l{i}.", layer.mixer, layer.mlp
        q = p + "mix."
        for n in ("norm1",) + (("norm2",) if f is not None else ()):
            plan.append((p + n, (w,), "gain", 0.1))
        if layer.type == "rglru":
            lin(q + "y", m.channels, w, True)
            lin(q + "x", m.channels, w, True)
            plan.append((q + "conv", (m.channels, m.conv), "normal", 1.0 / math.sqrt(m.conv)))
            plan.append((q + "conv.b", (m.channels,), "normal", 0.3))
            size = m.channels // m.blocks
            for n in ("ra", "ri"):
                plan.append((q + n, (m.blocks, size, size), "normal", 1.0 / math.sqrt(size)))
                plan.append((q + n + ".b", (m.blocks, size), "normal", 0.3))
            plan.append((q + "lam", (m.channels,), "around", -3.0))
            lin(q + "o", w, m.channels)
        elif layer.type == "latent_attention":
            lin(q + "dq", m.q_rank, w)
            plan.append((q + "dq.norm", (m.q_rank,), "gain", 0.1))
            lin(q + "uq", m.heads * (m.dim + m.rot_dim), m.q_rank)
            lin(q + "dkv", m.kv_rank + m.rot_dim, w)
            plan.append((q + "dkv.norm", (m.kv_rank,), "gain", 0.1))
            lin(q + "uk", m.heads * m.dim, m.kv_rank)
            lin(q + "uv", m.heads * m.vdim, m.kv_rank)
            lin(q + "o", w, m.heads * m.vdim)
        else:
            for n, heads in (("q", m.heads), ("k", m.kv_heads)):
                lin(q + n, heads * m.dim, w, True)
                plan.append((q + n + ".conv", (heads * m.dim, m.conv), "normal", 1.0 / math.sqrt(m.conv)))
                plan.append((q + n + ".norm", (m.dim,), "gain", 0.1))
            lin(q + "o", w, m.heads * m.dim)
        if f is not None:
            for name, ff in [(f"e{e}", f.ff) for e in range(f.experts)] + ([("shared", f.shared_ff)] if f.shared_ff else []):
                lin(f"{p}mlp.{name}.gate", ff, w)
                lin(f"{p}mlp.{name}.up", ff, w)
                lin(f"{p}mlp.{name}.down", w, ff)
            lin(p + "mlp.router", f.experts, w)
    plan.append(("final.norm", (w,), "gain", 0.1))
    return plan


register_architecture(Architecture(NAME, config_from_json, model_spec, init_plan, config_to_json))
