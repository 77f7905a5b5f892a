"""Ranudra: config.json keys, the model as specs, and checkpoint tensor names.

A decoder whose layers are listed one by one in ``layers``; each entry has a ``type`` (the mixer), the
mixer's sizes under ``mixer`` and its feed-forward under ``mlp`` (null: none).  The embedded tokens are
multiplied by ``embedding.scale``; the residual stream is kept in ``streams`` copies that every sublayer
reads and changes with learned coefficients (hyper-connections), in front of every sublayer a layer norm
(``norm.eps``, a weight, no bias).

* "latent_attention": attention over a cached latent of ``kv_rank`` numbers per token; a head of q has
  ``dim`` elements that meet keys made of the latent and ``rot_dim`` elements that, neighbours ``(2i, 2i +
  1)`` turned together by the position, meet one rotated key part shared by all heads; frequencies
  ``rot.base ** (-2i/dims)``, stretched by ``rot.scaling`` (factor, original, fast, slow) for long
  contexts; ``scale`` from the config; position ``i`` sees the last ``mask.size`` positions, itself
  included; values of ``vdim`` elements; every head's output times ``sigmoid(W_g h)`` of that head.
* "latent_attention_2": the same with a learned sink per head in the softmax's denominator and a gate per
  element of the concatenated heads.
* "gla": gated linear attention (:class:`~pylon_amd.config.specs.GatedLinearAttentionSpec`); the size
  between the two maps of its decays is the first one's number of rows.
* Feed-forward "dense": ``W_down relu(W_up h)^2``.

``loop`` names a stretch of layers ``start .. stop - 1`` that runs ``times`` times in a row over the same
weights, each pass with a cache or state of its own.  At the end the copies are summed; the head is the
embedding table, unscaled.

Keys that a mixer's entry leaves out switch the mechanism off: no ``rot``, no rotation; no
``rot.scaling``, plain frequencies; no ``mask``, every earlier key.  Without ``loop`` every layer runs once.

Tensors: ``embed``, ``final.norm``, per layer ``l<i>.norm1``, ``.norm2``, ``.hc1.{in,out,mix}``,
``.hc2.{in,out,mix}``; latent attention ``.mix.{q,dkv,uk,uv,g,o}``, ``.mix.dkv.norm`` and, of the second
kind, ``.mix.sink``; gla ``.mix.{q,k,v,g,a1,a2,o}``, ``.mix.a2.b``, ``.mix.norm``; feed-forward
``.mlp.{up,down}``.
"""
from __future__ import annotations

import math
from dataclasses import dataclass, replace
from typing import Dict, Mapping, Optional, Tuple

from ..config.registry import Architecture, WeightTarget, register_architecture
from ..config.specs import (
    GatedLinearAttentionSpec,
    LatentAttentionSpec,
    LayerSpec,
    ModelSpec,
    NormSpec,
    PlainFeedForwardSpec,
    PositionSpec,
    RotaryScalingSpec,
    ScheduleEntry,
)

ARCHITECTURE = "Ranudra"

DEFAULT_DECAY_RANK = 16  # for a configuration that comes without tensors (random weights) and names none


def _positive_int(value, name: str) -> int:
    if isinstance(value, bool) or not isinstance(value, int) or value < 1:
        raise ValueError(f"{name} must be a positive integer, got {value!r}")
    return value


def _positive(value, name: str) -> float:
    value = float(value)
    if not (value > 0 and math.isfinite(value)):
        raise ValueError(f"{name} must be positive and finite, got {value!r}")
    return value


def _require(data: Mapping, keys, where: str) -> None:
    missing = [key for key in keys if key not in data]
    if missing:
        raise ValueError(f"config.json lacks required keys in {where}: " + ", ".join(missing))


@dataclass(frozen=True)
class RotaryConfig:
    base: float
    dims: int
    scaling: Optional[Tuple[float, float, float, float]]  # factor, original, fast, slow


@dataclass(frozen=True)
class LatentConfig:
    heads: int
    dim: int
    rot_dim: int
    vdim: int
    kv_rank: int
    scale: float
    mask_size: Optional[int]
    rot: Optional[RotaryConfig]


@dataclass(frozen=True)
class LinearConfig:
    heads: int
    dim: int
    vdim: int
    tau: float
    decay_rank: Optional[int] = None  # None: not known yet (a tensor's shape gives it)


@dataclass(frozen=True)
class LayerConfig:
    type: str
    mixer: object  # LatentConfig or LinearConfig
    ff: Optional[int]  # hidden units of the feed-forward (None: the layer has none)


@dataclass(frozen=True)
class LoopConfig:
    start: int
    stop: int
    times: int


@dataclass(frozen=True)
class RanudraConfig:
    vocab: int
    width: int
    streams: int
    embedding_scale: float
    layers: Tuple[LayerConfig, ...]
    loop: Optional[LoopConfig]
    norm_eps: float
    initializer_range: float = 0.02  # only used to draw random weights
    eos_token_id: Optional[Tuple[int, ...]] = None

    def runs(self) -> Tuple[int, ...]:
        """The order in which the layers run."""
        count = len(self.layers)
        if self.loop is None:
            return tuple(range(count))
        start, stop = self.loop.start, self.loop.stop
        return (*range(start), *(tuple(range(start, stop)) * self.loop.times), *range(stop, count))


LATENT_TYPES = ("latent_attention", "latent_attention_2")


def _parse_rot(rot: Optional[Mapping], rot_dim: int, where: str) -> Optional[RotaryConfig]:
    if rot is None:
        return None
    _require(rot, ("base", "dims"), where)
    dims = _positive_int(rot["dims"], "rot.dims")
    if dims != rot_dim:
        raise ValueError(f"{where}: the whole rotated part turns, so rot.dims {dims} must equal rot_dim {rot_dim}")
    scaling = rot.get("scaling")
    if scaling is not None:
        _require(scaling, ("factor", "original", "fast", "slow"), where + ".scaling")
        scaling = tuple(_positive(scaling[key], f"rot.scaling.{key}") for key in ("factor", "original", "fast", "slow"))
    return RotaryConfig(_positive(rot["base"], "rot.base"), dims, scaling)


def _parse_mixer(kind: str, m: Mapping, where: str):
    if kind in LATENT_TYPES:
        _require(m, ("heads", "dim", "rot_dim", "vdim", "kv_rank", "scale"), where)
        rot_dim = _positive_int(m["rot_dim"], "rot_dim")
        if rot_dim % 2:
            raise ValueError(f"{where}: rot_dim {rot_dim} must be even")
        mask = m.get("mask")
        if mask is not None:
            _require(mask, ("size",), where + ".mask")
        return LatentConfig(
            _positive_int(m["heads"], "heads"), _positive_int(m["dim"], "dim"), rot_dim, _positive_int(m["vdim"], "vdim"),
            _positive_int(m["kv_rank"], "kv_rank"), _positive(m["scale"], "scale"),
            None if mask is None else _positive_int(mask["size"], "mask.size"), _parse_rot(m.get("rot"), rot_dim, where + ".rot"))
    if kind == "gla":
        _require(m, ("heads", "dim", "vdim", "tau"), where)
        rank = m.get("decay_rank")
        return LinearConfig(
            _positive_int(m["heads"], "heads"), _positive_int(m["dim"], "dim"), _positive_int(m["vdim"], "vdim"),
            _positive(m["tau"], "tau"), None if rank is None else _positive_int(rank, "decay_rank"))
    raise ValueError(f"{where}: unknown layer type {kind!r} (known: {', '.join(LATENT_TYPES)}, gla)")


def _parse_mlp(mlp: Optional[Mapping], where: str) -> Optional[int]:
    if mlp is None:
        return None
    _require(mlp, ("kind", "ff"), where)
    if mlp["kind"] != "dense":
        raise ValueError(f"{where}: unknown feed-forward kind {mlp['kind']!r} (known: dense)")
    return _positive_int(mlp["ff"], "ff")


def parse_config(data: Mapping) -> RanudraConfig:
    _require(data, ("vocab", "width", "streams", "embedding", "layers", "norm"), "the model")
    _require(data["norm"], ("eps",), "norm")
    _require(data["embedding"], ("scale",), "embedding")
    layers = []
    for index, entry in enumerate(data["layers"]):
        where = f"layers[{index}]"
        _require(entry, ("type", "mixer"), where)
        layers.append(LayerConfig(entry["type"], _parse_mixer(entry["type"], entry["mixer"], where + ".mixer"),
                                  _parse_mlp(entry.get("mlp"), where + ".mlp")))
    if not layers:
        raise ValueError("the model has no layers")
    loop = data.get("loop")
    if loop is not None:
        _require(loop, ("start", "stop", "times"), "loop")
        start, stop, times = int(loop["start"]), int(loop["stop"]), _positive_int(loop["times"], "loop.times")
        if not 0 <= start < stop <= len(layers):
            raise ValueError(f"loop: layers {start} .. {stop - 1} are not a stretch of the {len(layers)} layers")
        loop = LoopConfig(start, stop, times)
    eos = data.get("eos_token_id")
    if isinstance(eos, int):
        eos = (eos,)
    elif eos is not None:
        eos = tuple(int(v) for v in eos)
    return RanudraConfig(
        vocab=_positive_int(data["vocab"], "vocab"), width=_positive_int(data["width"], "width"),
        streams=_positive_int(data["streams"], "streams"), embedding_scale=float(data["embedding"]["scale"]),
        layers=tuple(layers), loop=loop, norm_eps=_positive(data["norm"]["eps"], "norm.eps"),
        initializer_range=float(data.get("initializer_range", 0.02)), eos_token_id=eos)


def with_tensor_shapes(cfg: RanudraConfig, shapes: Mapping[str, Tuple[int, ...]]) -> RanudraConfig:
    """The sizes that only a tensor's shape gives: the rows of every first map of the decays."""
    layers = []
    for index, layer in enumerate(cfg.layers):
        shape = shapes.get(f"l{index}.mix.a1")
        if isinstance(layer.mixer, LinearConfig) and shape is not None:
            layer = replace(layer, mixer=replace(layer.mixer, decay_rank=int(shape[0])))
        layers.append(layer)
    return replace(cfg, layers=tuple(layers))


def config_to_json(cfg: RanudraConfig) -> dict:
    layers = []
    for layer in cfg.layers:
        m = layer.mixer
        if isinstance(m, LinearConfig):
            mixer = {"heads": m.heads, "dim": m.dim, "vdim": m.vdim, "tau": m.tau}
            if m.decay_rank is not None:
                mixer["decay_rank"] = m.decay_rank
        else:
            mixer = {"heads": m.heads, "dim": m.dim, "rot_dim": m.rot_dim, "vdim": m.vdim, "kv_rank": m.kv_rank,
                     "scale": m.scale}
            if m.mask_size is not None:
                mixer["mask"] = {"size": m.mask_size}
            if m.rot is not None:
                mixer["rot"] = {"base": m.rot.base, "dims": m.rot.dims}
                if m.rot.scaling is not None:
                    mixer["rot"]["scaling"] = dict(zip(("factor", "original", "fast", "slow"), m.rot.scaling))
        layers.append({"type": layer.type, "mixer": mixer,
                       "mlp": None if layer.ff is None else {"kind": "dense", "ff": layer.ff}})
    out = {"architecture": ARCHITECTURE, "vocab": cfg.vocab, "width": cfg.width, "streams": cfg.streams,
           "embedding": {"scale": cfg.embedding_scale}, "layers": layers, "norm": {"eps": cfg.norm_eps},
           "initializer_range": cfg.initializer_range}
    if cfg.loop is not None:
        out["loop"] = {"start": cfg.loop.start, "stop": cfg.loop.stop, "times": cfg.loop.times}
    if cfg.eos_token_id is not None:
        out["eos_token_id"] = list(cfg.eos_token_id)
    return out


def _decay_rank(m: LinearConfig) -> int:
    return DEFAULT_DECAY_RANK if m.decay_rank is None else m.decay_rank


def _mixer_spec(cfg: RanudraConfig, layer: LayerConfig):
    m = layer.mixer
    if isinstance(m, LinearConfig):
        return GatedLinearAttentionSpec(
            hidden_size=cfg.width, n_heads=m.heads, head_dim=m.dim, v_head_dim=m.vdim, decay_rank=_decay_rank(m),
            tau=m.tau, norm_eps=cfg.norm_eps)
    second = layer.type == "latent_attention_2"
    position = None
    if m.rot is not None:
        scaling = None if m.rot.scaling is None else RotaryScalingSpec(*m.rot.scaling)
        position = PositionSpec(kind="rope", theta=m.rot.base, rotary_dim=m.rot.dims, interleaved=True, scaling=scaling)
    return LatentAttentionSpec(
        hidden_size=cfg.width, n_heads=m.heads, head_dim=m.dim, v_head_dim=m.vdim, q_rank=None, kv_rank=m.kv_rank,
        scale=m.scale, norm_eps=cfg.norm_eps, window=m.mask_size, gate=True, gate_over="element" if second else "head",
        rot_dim=m.rot_dim, position=position, sink=second)


def model_spec(cfg: RanudraConfig) -> ModelSpec:
    norm = NormSpec(kind="layernorm", dim=cfg.width, eps=cfg.norm_eps)
    layers = []
    for layer in cfg.layers:
        feed_forward = None
        if layer.ff is not None:
            feed_forward = PlainFeedForwardSpec(hidden_size=cfg.width, intermediate_size=layer.ff, activation="relu2")
        layers.append(LayerSpec(
            mixer=_mixer_spec(cfg, layer), feed_forward=feed_forward, mixer_norm=norm,
            feed_forward_norm=norm if feed_forward is not None else None, arrangement="hyper_connections",
            streams=cfg.streams))
    return ModelSpec(
        vocab_size=cfg.vocab, hidden_size=cfg.width, layers=tuple(layers),
        schedule=tuple(ScheduleEntry(layer=index) for index in cfg.runs()), final_norm=norm, tie_word_embeddings=True,
        max_positions=0, embedding_scale=cfg.embedding_scale, streams=cfg.streams)


def _latent_targets(targets: Dict[str, WeightTarget], src: str, dst: str, m: LatentConfig, width: int, second: bool) -> None:
    q, vv = m.heads * (m.dim + m.rot_dim), m.heads * m.vdim
    latent = m.kv_rank + m.rot_dim
    # the projections that read the mixer's input are rows of one matrix
    targets[f"{src}.q"] = WeightTarget(f"{dst}.down", (q, width), 0)
    targets[f"{src}.dkv"] = WeightTarget(f"{dst}.down", (latent, width), q)
    targets[f"{src}.g"] = WeightTarget(f"{dst}.down", (vv if second else m.heads, width), q + latent)
    targets[f"{src}.dkv.norm"] = WeightTarget(f"{dst}.c_norm", (m.kv_rank,), role="vector", init="ones_jitter")
    targets[f"{src}.uk"] = WeightTarget(f"{dst}.uk", (m.heads * m.dim, m.kv_rank))
    targets[f"{src}.uv"] = WeightTarget(f"{dst}.uv", (vv, m.kv_rank))
    targets[f"{src}.o"] = WeightTarget(f"{dst}.out", (width, vv))
    if second:
        targets[f"{src}.sink"] = WeightTarget(f"{dst}.sink", (m.heads,), role="vector")


def _linear_targets(targets: Dict[str, WeightTarget], src: str, dst: str, m: LinearConfig, width: int) -> None:
    qk, vv, rank = m.heads * m.dim, m.heads * m.vdim, _decay_rank(m)
    start = 0
    for name, rows in (("q", qk), ("k", qk), ("v", vv), ("g", vv), ("a1", rank)):
        targets[f"{src}.{name}"] = WeightTarget(f"{dst}.proj", (rows, width), start)
        start += rows
    targets[f"{src}.a2"] = WeightTarget(f"{dst}.a2", (qk, rank), role="vector")
    targets[f"{src}.a2.b"] = WeightTarget(f"{dst}.a2_bias", (qk,), role="vector")
    targets[f"{src}.norm"] = WeightTarget(f"{dst}.norm", (m.vdim,), role="vector", init="ones_jitter")
    targets[f"{src}.o"] = WeightTarget(f"{dst}.out", (width, vv))


def weight_targets(cfg: RanudraConfig) -> Dict[str, WeightTarget]:
    width, streams = cfg.width, cfg.streams
    norm = dict(role="vector", init="ones_jitter")
    targets: Dict[str, WeightTarget] = {
        "embed": WeightTarget("embed", (cfg.vocab, width)),
        "final.norm": WeightTarget("final_norm.weight", (width,), **norm),
    }
    for index, layer in enumerate(cfg.layers):
        src, dst = f"l{index}", f"layers.{index}"
        if isinstance(layer.mixer, LinearConfig):
            _linear_targets(targets, f"{src}.mix", f"{dst}.mixer", layer.mixer, width)
        else:
            _latent_targets(targets, f"{src}.mix", f"{dst}.mixer", layer.mixer, width, layer.type == "latent_attention_2")
        parts = [("1", "mixer")] + ([("2", "feed_forward")] if layer.ff is not None else [])
        for number, part in parts:
            targets[f"{src}.norm{number}"] = WeightTarget(f"{dst}.{part}_norm.weight", (width,), **norm)
            targets[f"{src}.hc{number}.in"] = WeightTarget(f"{dst}.{part}_read", (streams,), role="vector", init="ones_jitter")
            targets[f"{src}.hc{number}.out"] = WeightTarget(f"{dst}.{part}_write", (streams,), role="vector", init="ones_jitter")
            targets[f"{src}.hc{number}.mix"] = WeightTarget(f"{dst}.{part}_mix", (streams, streams), role="vector")
        if layer.ff is not None:
            targets[f"{src}.mlp.up"] = WeightTarget(f"{dst}.feed_forward.up", (layer.ff, width))
            targets[f"{src}.mlp.down"] = WeightTarget(f"{dst}.feed_forward.down", (width, layer.ff))
    return targets


RANUDRA = register_architecture(
    Architecture(
        name=ARCHITECTURE,
        parse_config=parse_config,
        model_spec=model_spec,
        weight_targets=weight_targets,
        config_to_json=config_to_json,
        with_tensor_shapes=with_tensor_shapes,
    ),
    replace=True,
)
