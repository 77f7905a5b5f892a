"""Tiny Ranudra configurations for the tests, and model folders made from them."""
from __future__ import annotations

import json
from pathlib import Path

import numpy as np


def _rot(base, dims, scaling=None):
    out = {"base": base, "dims": dims}
    if scaling is not None:
        out["scaling"] = dict(zip(("factor", "original", "fast", "slow"), scaling))
    return out


def _latent(heads, dim, rot_dim, vdim, kv_rank, scale, rot=None, size=None):
    out = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank, "scale": scale}
    if rot is not None:
        out["rot"] = rot
    if size is not None:
        out["mask"] = {"size": size}
    return out


def _gla(heads, dim, vdim, tau, rank=None):
    out = {"heads": heads, "dim": dim, "vdim": vdim, "tau": tau}
    if rank is not None:
        out["decay_rank"] = rank
    return out


def _layer(kind, mixer, ff):
    return {"type": kind, "mixer": mixer, "mlp": None if ff is None else {"kind": "dense", "ff": ff}}


def _model(vocab, width, streams, scale, eps, layers, loop=None):
    out = {"architecture": "Ranudra", "vocab": vocab, "width": width, "streams": streams, "embedding": {"scale": scale},
           "norm": {"eps": eps}, "layers": layers}
    if loop is not None:
        out["loop"] = dict(zip(("start", "stop", "times"), loop))
    return out


# A: sizes that are no multiples of 8 (the general kernels everywhere), windows of a few positions (every
# prompt crosses many edges), three copies of the stream, a looped stretch in the middle, a layer without
# feed-forward, values smaller and larger than keys.
RANUDRA_A = _model(113, 40, 3, 5.0, 2e-5, [
    _layer("latent_attention_2", _latent(3, 6, 10, 4, 12, 0.45, _rot(300.0, 10), 13), 28),
    _layer("gla", _gla(3, 12, 20, 4.0, 5), None),
    _layer("latent_attention", _latent(5, 10, 6, 14, 18, 0.4, _rot(5000.0, 6, (4.0, 16, 4.0, 1.0)), 7), 36),
    _layer("gla", _gla(2, 20, 6, 11.0, 3), 20),
], (1, 3, 2))
# B: rows that the matrix-core kernels take with room (80 of 96 and 128 elements), windows that are no
# multiple of a page or a block, linear attention first and last, two copies, the loop at the end.
RANUDRA_B = _model(160, 64, 2, 8.0, 1e-6, [
    _layer("gla", _gla(2, 32, 64, 10.0), 88),
    _layer("latent_attention", _latent(6, 32, 16, 48, 64, 0.17, _rot(8.0e5, 16, (6.0, 64, 16.0, 2.0)), 50), 72),
    _layer("latent_attention_2", _latent(8, 16, 32, 24, 96, 0.2, _rot(3.0e5, 32), 100), 96),
    _layer("gla", _gla(4, 16, 32, 9.0, 8), 64),
], (2, 4, 3))
# C: more than 16 heads, a row of 256 + 64 elements and one of 128 + 32 that sees every earlier key, four
# copies, the whole model looped, a decay taken as it is (tau 1).
RANUDRA_C = _model(97, 128, 4, 3.0, 3e-6, [
    _layer("latent_attention", _latent(20, 24, 64, 16, 256, 0.12, _rot(1.0e4, 64, (2.0, 32, 8.0, 1.0)), 129), 112),
    _layer("gla", _gla(2, 64, 128, 1.0, 16), 128),
    _layer("latent_attention_2", _latent(17, 40, 32, 24, 128, 0.13, _rot(7.0e4, 32)), 104),
], (0, 3, 2))
# D: one copy, no loop, a window of one page, one of one key, an unrotated part, linear heads of 128 x 32
# and 256 x 24.
RANUDRA_D = _model(203, 96, 1, 11.0, 1e-5, [
    _layer("gla", _gla(2, 128, 32, 8.0, 24), None),
    _layer("latent_attention", _latent(4, 32, 64, 40, 192, 0.15, _rot(1.0e5, 64), 64), 80),
    _layer("latent_attention_2", _latent(4, 24, 8, 56, 40, 0.3, None, 1), 48),
    _layer("gla", _gla(1, 256, 24, 20.0, 2), 160),
])
# E: a width of 100, a vocabulary of 301, the widest rows (512 + 64), strong decays (tau 0.5).
RANUDRA_E = _model(301, 100, 2, 14.0, 1e-6, [
    _layer("latent_attention_2", _latent(2, 20, 64, 12, 512, 0.1, _rot(1.0e4, 64), 90), 60),
    _layer("gla", _gla(3, 32, 48, 0.5, 4), 44),
    _layer("latent_attention", _latent(3, 12, 4, 10, 28, 0.3, _rot(777.0, 4, (3.0, 20, 5.0, 1.0)), 9), 52),
], (1, 2, 4))
CONFIGS = {"A": RANUDRA_A, "B": RANUDRA_B, "C": RANUDRA_C, "D": RANUDRA_D, "E": RANUDRA_E}


def make_folder(tmp: Path, name: str, *, dtype: str = "float32", seed: int = 5, std: float = 0.12, config=None) -> Path:
    """A model folder of random weights changed after drawing so that faults show: sinks as large as
    scores, decays close to one (a lost state is missed for many tokens), copies of the stream that mix
    but do not fade, norm weights and shares that differ from one and from each other."""
    import torch
    from safetensors.torch import load_file, save_file

    from pylon_amd.weights import write_random_model

    folder = write_random_model(Path(tmp) / f"ranudra_{name}_{dtype}_{seed}", config or CONFIGS[name], seed,
                                dtype=dtype, std=std, norm_jitter=0.2)
    path = folder / "model.safetensors"
    tensors = load_file(str(path))
    for key in list(tensors):
        value = tensors[key].float()
        if key.endswith(".mix.k"):
            # keys that lie close to their queries: the read-out of a head is normed, so where its products
            # nearly cancel (a first token whose q and k are orthogonal) rounding alone decides its sign
            value = 0.7 * tensors[key[:-1] + "q"].float() + 0.5 * value
        elif key.endswith(".sink"):
            value = value * 12.0
        elif key.endswith(".a2.b"):
            value = value * 8.0 + 2.5
        elif key.endswith((".hc1.mix", ".hc2.mix")):
            value = torch.eye(len(value)) + value * 2.0
        elif key.endswith((".hc1.in", ".hc2.in")):
            value = value / len(value)
        elif key.endswith(".mix.dkv"):
            value = value * 1.5
        else:
            continue
        tensors[key] = value.to(tensors[key].dtype)
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
