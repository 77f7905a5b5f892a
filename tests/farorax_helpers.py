"""Tiny Farorax configurations for the tests, and model folders made from them."""
from __future__ import annotations

import json
from pathlib import Path

import numpy as np


def _rot(base, dims, scaling=None):
    out = {"base": base, "dims": dims}
    if scaling is not None:
        out["scaling"] = dict(zip(("factor", "low", "high", "original"), scaling))
    return out


def _attention(heads, kv_heads, dim, vdim, scale, rot=None, size=None):
    out = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale}
    if rot is not None:
        out["rot"] = rot
    if size is not None:
        out["mask"] = {"size": size}
    return out


def _lightning(heads, dim, vdim, decay=None):
    if decay is None:
        decay = np.linspace(0.55, 0.997, heads).round(4).tolist()
    return {"heads": heads, "dim": dim, "vdim": vdim, "decay": list(decay)}


def _dense(ff):
    return {"kind": "dense", "ff": ff}


def _moe(experts, top, ff, groups=None, shared=None):
    out = {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}
    if groups is not None:
        out["router"]["groups"] = dict(zip(("count", "keep"), groups))
    if shared is not None:
        out["shared"] = {"ff": shared}
    return out


def _layer(mixer, mlp):
    return {"type": "lightning" if "decay" in mixer else "attention", "mixer": mixer, "mlp": mlp}


def _model(vocab, width, eps, layers, *, loop=None, mult=1.0, cap=None):
    out = {"architecture": "Farorax", "vocab": vocab, "width": width, "norm": {"eps": eps}, "residual_mult": mult,
           "layers": layers}
    if loop is not None:
        out["loop"] = dict(zip(("start", "stop", "times"), loop))
    if cap is not None:
        out["logit_softcap"] = cap
    return out


# A: sizes that are no multiples of 8 (the general kernels everywhere), windows of a few positions, a looped
# stretch in the middle, a layer without feed-forward, values smaller and larger than keys.
FARORAX_A = _model(113, 40, 2e-5, [
    _layer(_lightning(3, 12, 20), _dense(28)),
    _layer(_attention(4, 2, 10, 14, 0.4, _rot(500.0, 6, (4.0, 1.0, 4.0, 24)), 7), _moe(6, 2, 16, (3, 2), 12)),
    _layer(_lightning(2, 20, 6), None),
    _layer(_attention(3, 3, 12, 8, 0.3, _rot(1.0e4, 12), 5), _dense(20)),
], loop=(1, 3, 2), mult=0.7, cap=15.0)
# B: sizes that the matrix-core kernels take, windows that are no multiple of a page or a block of keys, the
# loop at the end with three passes, the sorted expert path, groups of which one or half are kept.
FARORAX_B = _model(160, 64, 1e-6, [
    _layer(_lightning(2, 32, 64), _moe(8, 3, 24, (4, 2))),
    _layer(_attention(6, 2, 64, 48, 0.15, _rot(8.0e4, 32, (8.0, 1.5, 5.0, 128)), 50), _dense(88)),
    _layer(_lightning(4, 64, 32), _dense(72)),
    _layer(_attention(3, 3, 32, 64, 0.2, _rot(3.0e5, 32, (2.0, 1.0, 8.0, 64)), 100), _moe(12, 4, 40, (2, 1), 56)),
], loop=(2, 4, 3), mult=0.45, cap=25.0)
# C: heads of 128 on both sides, eight query heads on one key/value head, a window longer than any prompt, the
# whole model looped, no groups, one expert of four a token, two experts of which both run.
FARORAX_C = _model(97, 128, 3e-6, [
    _layer(_attention(8, 1, 128, 128, 0.09, _rot(2.0e4, 64, (16.0, 1.0, 2.0, 512)), 1000), _moe(4, 1, 64, None, 32)),
    _layer(_lightning(2, 128, 128, (0.9, 0.999)), _moe(2, 2, 40)),
], loop=(0, 2, 2), mult=0.8)
# D: no loop, no cap, sublayers added as they are; a window of one page, one of one key, one attention that
# sees everything; no rotation, or a small part rotated; linear heads of 256 x 24 and 8 x 200.
FARORAX_D = _model(203, 96, 1e-5, [
    _layer(_lightning(1, 256, 24, (0.98,)), None),
    _layer(_attention(4, 2, 40, 72, 0.16, None, 64), _moe(9, 4, 32, (3, 2))),
    _layer(_lightning(5, 8, 200), _dense(160)),
    _layer(_attention(2, 2, 24, 24, 0.2, _rot(1.0e5, 8), 1), _dense(48)),
    _layer(_attention(4, 1, 16, 32, 0.25, _rot(1.0e4, 16, (4.0, 1.0, 4.0, 40))), None),
])
# E: a width of 100, a vocabulary of 301; groups of one expert each; decays of nothing, a half and one; a loop of
# one pass.
FARORAX_E = _model(301, 100, 1e-6, [
    _layer(_attention(5, 5, 12, 10, 0.3, _rot(777.0, 12, (3.0, 2.0, 6.0, 20)), 9), _moe(5, 3, 20, (5, 4), 12)),
    _layer(_lightning(3, 10, 6, (0.0, 0.5, 1.0)), _moe(11, 5, 12)),
], loop=(0, 1, 1), mult=0.25, cap=4.0)
CONFIGS = {"A": FARORAX_A, "B": FARORAX_B, "C": FARORAX_C, "D": FARORAX_D, "E": FARORAX_E}


def make_folder(tmp: Path, name: str, *, dtype: str = "float32", seed: int = 5, std: float = 0.12,
                router_scale: float = 2.5, config=None) -> Path:
    """A model folder of random weights changed after drawing so that faults show: routers scaled up (clear
    choices: the tests do not rest on close calls), sinks as large as scores, passes that begin with vectors
    of their own as large as the stream, norm weights that differ from one."""
    from safetensors.torch import load_file, save_file

    from pylon_amd.weights import write_random_model

    folder = write_random_model(Path(tmp) / f"farorax_{name}_{dtype}_{seed}", config or CONFIGS[name], seed,
                                dtype=dtype, std=std, norm_jitter=0.2)
    path = folder / "model.safetensors"
    tensors = load_file(str(path))
    for key in list(tensors):
        factor = {"router": router_scale, "sink": 12.0, "step": 4.0, "embed": 4.0}.get(key.rsplit(".", 1)[-1])
        if factor is not None:
            tensors[key] = (tensors[key].float() * factor).to(tensors[key].dtype)
    save_file(tensors, str(path))
    return folder


def read_folder(folder: Path):
    import torch
    from safetensors.torch import load_file

    cfg = json.loads((Path(folder) / "config.json").read_text())
    weights = {name: t.to(torch.float64).numpy() for name, t in load_file(str(Path(folder) / "model.safetensors")).items()}
    return cfg, weights


def tokens(vocab: int, count: int, seed: int):
    return np.random.default_rng(seed).integers(0, vocab, count).tolist()
