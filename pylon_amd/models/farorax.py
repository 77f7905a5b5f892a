"""Farorax: config.json keys, the model as specs, and checkpoint tensor names.

A decoder whose layers are listed one by one in ``layers``; each entry has a ``type`` (the mixer:
"attention" or "lightning"), the mixer's sizes under ``mixer`` and its feed-forward under ``mlp``
(null: none).  A layer is pre-normed (RMS norms with ``norm.eps``), and both its sublayers' outputs are
multiplied by ``residual_mult`` as they are added to the stream.

* "attention": grouped queries with keys of ``dim`` and values of ``vdim`` elements; neighbours ``(2i, 2i +
  1)`` of the first ``rot.dims`` elements of every head of q and k turn together, with frequencies
  ``rot.base ** (-2i/dims)`` that ``rot.scaling`` (factor, low, high, original) stretches by wavelength;
  ``scale`` from the config; a sliding window of ``mask.size`` keys; a learned sink per head in the
  softmax's denominator.
* "lightning": linear attention with a fixed ``decay`` per head on activated projections, normed over
  all heads and gated (:class:`~pylon_amd.config.specs.LightningAttentionSpec`).
* Feed-forward "dense": gated through gelu's tanh form.  "moe": ``router.experts`` experts of
  ``expert.ff`` hidden units gated through silu, scored by the sigmoids of the router's outputs; of
  ``router.groups.count`` groups of neighbouring experts the ``keep`` with the largest sums of their two
  best scores can be chosen from; a token takes the ``top`` best, weighted by their scores over the scores'
  sum; a shared expert of ``shared.ff`` hidden units runs for every token.
* ``loop``: layers ``start .. stop - 1`` run ``times`` times in a row over the same weights, each pass with
  caches and states of its own; ahead of every pass the stream and the embedded tokens go through one
  matrix together and the pass's own vector is added.
* The final norm, the head (a matrix of its own), logits soft-capped at ``logit_softcap``.

Keys that an entry leaves out switch the mechanism off: no ``rot``, no rotation; no ``rot.scaling``, plain
frequencies; no ``mask``, every earlier key; no ``groups``, one group; no ``shared``, no shared expert; no
``loop``, ``logit_softcap`` or ``residual_mult``.

Tensors: ``embed``, ``head``, ``final.norm``, ``loop.in``, ``loop.step``, per layer ``l<i>.norm1``,
``.norm2``; attention ``.mix.{q,k,v,o,sink}``; lightning ``.mix.{q,k,v,g,o,norm}``; dense
``.mlp.{gate,up,down}``; mixture ``.mlp.e<j>.{gate,up,down}``, ``.mlp.router``, ``.mlp.shared.{gate,up,down}``.
"""
from __future__ import annotations

import math
from dataclasses import dataclass
from typing import Dict, Mapping, Optional, Tuple

from ..config.registry import Architecture, WeightTarget, register_architecture
from ..config.specs import (
    AttentionSpec,
    GatedFeedForwardSpec,
    LayerSpec,
    LightningAttentionSpec,
    LogitSoftcapSpec,
    MixtureFeedForwardSpec,
    ModelSpec,
    NormSpec,
    PassEntrySpec,
    PositionSpec,
    RotaryBandScalingSpec,
    ScheduleEntry,
)

ARCHITECTURE = "Farorax"

_SCALING_KEYS = ("factor", "low", "high", "original")


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
    scaling: Optional[Tuple[float, float, float, float]]  # factor, low, high, original


@dataclass(frozen=True)
class AttentionConfig:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    rot: Optional[RotaryConfig]
    mask_size: Optional[int]


@dataclass(frozen=True)
class LightningConfig:
    heads: int
    dim: int
    vdim: int
    decay: Tuple[float, ...]


@dataclass(frozen=True)
class DenseConfig:
    ff: int


@dataclass(frozen=True)
class MixtureConfig:
    experts: int
    top: int
    ff: int
    groups: int
    keep: int
    shared_ff: Optional[int]


@dataclass(frozen=True)
class LayerConfig:
    type: str
    mixer: object  # AttentionConfig or LightningConfig
    mlp: Optional[object]  # DenseConfig or MixtureConfig


@dataclass(frozen=True)
class LoopConfig:
    start: int
    stop: int
    times: int


@dataclass(frozen=True)
class FaroraxConfig:
    vocab: int
    width: int
    layers: Tuple[LayerConfig, ...]
    loop: Optional[LoopConfig]
    norm_eps: float
    residual_mult: float
    logit_softcap: Optional[float]
    initializer_range: float = 0.02  # only used to draw random weights
    eos_token_id: Optional[Tuple[int, ...]] = None

    def runs(self) -> Tuple[Tuple[int, Optional[int]], ...]:
        """The order in which the layers run: ``(layer, number of the pass that begins right before it)``."""
        count = len(self.layers)
        if self.loop is None:
            return tuple((i, None) for i in range(count))
        loop = self.loop
        order = [(i, None) for i in range(loop.start)]
        for t in range(loop.times):
            order += [(i, t if i == loop.start else None) for i in range(loop.start, loop.stop)]
        return tuple(order + [(i, None) for i in range(loop.stop, count)])


def _parse_rot(rot: Optional[Mapping], dim: int, where: str) -> Optional[RotaryConfig]:
    if rot is None:
        return None
    _require(rot, ("base", "dims"), where)
    dims = rot["dims"]
    if dims == 0:
        return None
    dims = _positive_int(dims, "rot.dims")
    if dims % 2 or dims > dim:
        raise ValueError(f"{where}: rot.dims {dims} must be even and at most the head's {dim} elements")
    scaling = rot.get("scaling")
    if scaling is not None:
        _require(scaling, _SCALING_KEYS, where + ".scaling")
        scaling = tuple(_positive(scaling[key], f"rot.scaling.{key}") for key in _SCALING_KEYS)
        if not scaling[1] < scaling[2]:
            raise ValueError(f"{where}.scaling: low {scaling[1]} must be less than high {scaling[2]}")
    return RotaryConfig(_positive(rot["base"], "rot.base"), dims, scaling)


def _parse_mixer(kind: str, m: Mapping, where: str):
    if kind == "attention":
        _require(m, ("heads", "kv_heads", "dim", "vdim", "scale"), where)
        heads, kv_heads = _positive_int(m["heads"], "heads"), _positive_int(m["kv_heads"], "kv_heads")
        if heads % kv_heads:
            raise ValueError("The number of Q heads must be divisible by the number of KV heads.")
        dim = _positive_int(m["dim"], "dim")
        mask, size = m.get("mask"), None
        if mask is not None:
            _require(mask, ("size",), where + ".mask")
            size = _positive_int(mask["size"], "mask.size")
        return AttentionConfig(heads, kv_heads, dim, _positive_int(m["vdim"], "vdim"), _positive(m["scale"], "scale"),
                               _parse_rot(m.get("rot"), dim, where + ".rot"), size)
    if kind == "lightning":
        _require(m, ("heads", "dim", "vdim", "decay"), where)
        heads = _positive_int(m["heads"], "heads")
        decay = tuple(float(d) for d in m["decay"])
        if len(decay) != heads or not all(0.0 <= d <= 1.0 for d in decay):
            raise ValueError(f"{where}: decay must hold {heads} numbers from 0 to 1, got {list(decay)}")
        return LightningConfig(heads, _positive_int(m["dim"], "dim"), _positive_int(m["vdim"], "vdim"), decay)
    raise ValueError(f"{where}: unknown layer type {kind!r} (known: attention, lightning)")


def _parse_mlp(mlp: Optional[Mapping], where: str):
    if mlp is None:
        return None
    _require(mlp, ("kind",), where)
    if mlp["kind"] == "dense":
        _require(mlp, ("ff",), where)
        return DenseConfig(_positive_int(mlp["ff"], "ff"))
    if mlp["kind"] != "moe":
        raise ValueError(f"{where}: unknown feed-forward kind {mlp['kind']!r} (known: dense, moe)")
    _require(mlp, ("expert", "router"), where)
    _require(mlp["expert"], ("ff",), where + ".expert")
    router = mlp["router"]
    _require(router, ("experts", "top"), where + ".router")
    experts, top = _positive_int(router["experts"], "experts"), _positive_int(router["top"], "top")
    groups, keep = 1, 1
    if router.get("groups") is not None:
        _require(router["groups"], ("count", "keep"), where + ".router.groups")
        groups = _positive_int(router["groups"]["count"], "groups.count")
        keep = _positive_int(router["groups"]["keep"], "groups.keep")
    if experts % groups or keep > groups:
        raise ValueError(f"{where}: {experts} experts do not form {groups} equal groups of which {keep} are kept")
    if top > experts // groups * keep:
        raise ValueError(f"{where}: top {top} exceeds the {experts // groups * keep} experts of the kept groups")
    shared = mlp.get("shared")
    if shared is not None:
        _require(shared, ("ff",), where + ".shared")
        shared = _positive_int(shared["ff"], "shared.ff")
    return MixtureConfig(experts, top, _positive_int(mlp["expert"]["ff"], "expert.ff"), groups, keep, shared)


def parse_config(data: Mapping) -> FaroraxConfig:
    _require(data, ("vocab", "width", "layers", "norm"), "the model")
    _require(data["norm"], ("eps",), "norm")
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
    mult = float(data.get("residual_mult", 1.0))
    if not math.isfinite(mult):
        raise ValueError(f"residual_mult must be finite, got {mult!r}")
    cap = data.get("logit_softcap")
    eos = data.get("eos_token_id")
    if isinstance(eos, int):
        eos = (eos,)
    elif eos is not None:
        eos = tuple(int(v) for v in eos)
    return FaroraxConfig(
        vocab=_positive_int(data["vocab"], "vocab"), width=_positive_int(data["width"], "width"),
        layers=tuple(layers), loop=loop, norm_eps=_positive(data["norm"]["eps"], "norm.eps"), residual_mult=mult,
        logit_softcap=None if cap is None else _positive(cap, "logit_softcap"),
        initializer_range=float(data.get("initializer_range", 0.02)), eos_token_id=eos)


def _mixer_json(m) -> dict:
    if isinstance(m, LightningConfig):
        return {"heads": m.heads, "dim": m.dim, "vdim": m.vdim, "decay": list(m.decay)}
    out = {"heads": m.heads, "kv_heads": m.kv_heads, "dim": m.dim, "vdim": m.vdim, "scale": m.scale}
    if m.rot is not None:
        out["rot"] = {"base": m.rot.base, "dims": m.rot.dims}
        if m.rot.scaling is not None:
            out["rot"]["scaling"] = dict(zip(_SCALING_KEYS, m.rot.scaling))
    if m.mask_size is not None:
        out["mask"] = {"size": m.mask_size}
    return out


def _mlp_json(f) -> Optional[dict]:
    if f is None:
        return None
    if isinstance(f, DenseConfig):
        return {"kind": "dense", "ff": f.ff}
    router = {"experts": f.experts, "top": f.top}
    if f.groups != 1:
        router["groups"] = {"count": f.groups, "keep": f.keep}
    out = {"kind": "moe", "expert": {"ff": f.ff}, "router": router}
    if f.shared_ff is not None:
        out["shared"] = {"ff": f.shared_ff}
    return out


def config_to_json(cfg: FaroraxConfig) -> dict:
    out = {"architecture": ARCHITECTURE, "vocab": cfg.vocab, "width": cfg.width,
           "layers": [{"type": layer.type, "mixer": _mixer_json(layer.mixer), "mlp": _mlp_json(layer.mlp)}
                      for layer in cfg.layers],
           "norm": {"eps": cfg.norm_eps}, "residual_mult": cfg.residual_mult, "initializer_range": cfg.initializer_range}
    if cfg.loop is not None:
        out["loop"] = {"start": cfg.loop.start, "stop": cfg.loop.stop, "times": cfg.loop.times}
    if cfg.logit_softcap is not None:
        out["logit_softcap"] = cfg.logit_softcap
    if cfg.eos_token_id is not None:
        out["eos_token_id"] = list(cfg.eos_token_id)
    return out


def _mixer_spec(cfg: FaroraxConfig, m):
    if isinstance(m, LightningConfig):
        return LightningAttentionSpec(hidden_size=cfg.width, n_heads=m.heads, head_dim=m.dim, v_head_dim=m.vdim,
                                      decay=m.decay, norm_eps=cfg.norm_eps)
    position = PositionSpec(kind="none")
    if m.rot is not None:
        scaling = None if m.rot.scaling is None else RotaryBandScalingSpec(*m.rot.scaling)
        position = PositionSpec(kind="rope", theta=m.rot.base, rotary_dim=m.rot.dims, interleaved=True, scaling=scaling)
    return AttentionSpec(hidden_size=cfg.width, n_heads=m.heads, n_kv_heads=m.kv_heads, head_dim=m.dim, scale=m.scale,
                         position=position, qk_norm=False, v_head_dim=m.vdim, window=m.mask_size, sink=True)


def _feed_forward_spec(cfg: FaroraxConfig, f):
    if f is None:
        return None
    if isinstance(f, DenseConfig):
        return GatedFeedForwardSpec(hidden_size=cfg.width, intermediate_size=f.ff, activation="gelu_tanh")
    return MixtureFeedForwardSpec(
        hidden_size=cfg.width, n_experts=f.experts, top=f.top, expert_size=f.ff, shared_size=f.shared_ff,
        shared_gate=False, router_bias=False, scoring="sigmoid", groups=f.groups, groups_kept=f.keep,
        group_score="top2", renormalize=True)


def model_spec(cfg: FaroraxConfig) -> ModelSpec:
    norm = NormSpec(kind="rmsnorm", dim=cfg.width, eps=cfg.norm_eps)
    layers = []
    for layer in cfg.layers:
        feed_forward = _feed_forward_spec(cfg, layer.mlp)
        layers.append(LayerSpec(
            mixer=_mixer_spec(cfg, layer.mixer), feed_forward=feed_forward, mixer_norm=norm,
            feed_forward_norm=norm if feed_forward is not None else None, arrangement="pre_norm",
            residual_factor=cfg.residual_mult))
    schedule = tuple(ScheduleEntry(layer=index, begins_pass=t) for index, t in cfg.runs())
    return ModelSpec(
        vocab_size=cfg.vocab, hidden_size=cfg.width, layers=tuple(layers), schedule=schedule, final_norm=norm,
        tie_word_embeddings=False, max_positions=0,
        logit_parts=(LogitSoftcapSpec(cap=cfg.logit_softcap),) if cfg.logit_softcap is not None else (),
        pass_entry=PassEntrySpec(dim=cfg.width, times=cfg.loop.times) if cfg.loop is not None else None)


def _stacked(targets: Dict[str, WeightTarget], src: str, param: str, rows: Mapping[str, int], width: int,
             start: int = 0) -> None:
    """Projections of one input as the rows of one matrix, in the order given."""
    for name, count in rows.items():
        targets[f"{src}.{name}"] = WeightTarget(param, (count, width), start)
        start += count


def weight_targets(cfg: FaroraxConfig) -> Dict[str, WeightTarget]:
    width = cfg.width
    around_one = dict(role="vector", init="ones_jitter")
    targets: Dict[str, WeightTarget] = {
        "embed": WeightTarget("embed", (cfg.vocab, width)),
        "head": WeightTarget("lm_head", (cfg.vocab, width)),
        "final.norm": WeightTarget("final_norm.weight", (width,), **around_one),
    }
    if cfg.loop is not None:
        targets["loop.in"] = WeightTarget("pass_entry.join", (width, 2 * width))
        targets["loop.step"] = WeightTarget("pass_entry.step", (cfg.loop.times, width), role="vector")
    for index, layer in enumerate(cfg.layers):
        src, dst = f"l{index}", f"layers.{index}"
        m, mix = layer.mixer, f"{dst}.mixer"
        targets[f"{src}.norm1"] = WeightTarget(f"{dst}.mixer_norm.weight", (width,), **around_one)
        if isinstance(m, LightningConfig):
            qk, vg = m.heads * m.dim, m.heads * m.vdim
            _stacked(targets, f"{src}.mix", f"{mix}.qkvg", {"q": qk, "k": qk, "v": vg, "g": vg}, width)
            targets[f"{src}.mix.norm"] = WeightTarget(f"{mix}.norm", (vg,), **around_one)
            targets[f"{src}.mix.o"] = WeightTarget(f"{mix}.out", (width, vg))
        else:
            _stacked(targets, f"{src}.mix", f"{mix}.qkv",
                     {"q": m.heads * m.dim, "k": m.kv_heads * m.dim, "v": m.kv_heads * m.vdim}, width)
            targets[f"{src}.mix.sink"] = WeightTarget(f"{mix}.sink", (m.heads,), role="vector")
            targets[f"{src}.mix.o"] = WeightTarget(f"{mix}.out", (width, m.heads * m.vdim))
        f, ffn = layer.mlp, f"{dst}.feed_forward"
        if f is None:
            continue
        targets[f"{src}.norm2"] = WeightTarget(f"{dst}.feed_forward_norm.weight", (width,), **around_one)
        if isinstance(f, DenseConfig):
            _stacked(targets, f"{src}.mlp", f"{ffn}.gate_up", {"gate": f.ff, "up": f.ff}, width)
            targets[f"{src}.mlp.down"] = WeightTarget(f"{ffn}.down", (width, f.ff))
            continue
        targets[f"{src}.mlp.router"] = WeightTarget(f"{ffn}.router", (f.experts, width))
        for e in range(f.experts):
            _stacked(targets, f"{src}.mlp.e{e}", f"{ffn}.gate_up", {"gate": f.ff, "up": f.ff}, width, e * 2 * f.ff)
            targets[f"{src}.mlp.e{e}.down"] = WeightTarget(f"{ffn}.down", (width, f.ff), e * width)
        if f.shared_ff is not None:
            _stacked(targets, f"{src}.mlp.shared", f"{ffn}.shared_gate_up", {"gate": f.shared_ff, "up": f.shared_ff}, width)
            targets[f"{src}.mlp.shared.down"] = WeightTarget(f"{ffn}.shared_down", (width, f.shared_ff))
    return targets


FARORAX = register_architecture(
    Architecture(
        name=ARCHITECTURE,
        parse_config=parse_config,
        model_spec=model_spec,
        weight_targets=weight_targets,
        config_to_json=config_to_json,
    ),
    replace=True,
)
