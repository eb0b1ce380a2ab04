"""Tiny Semezen configurations for tests; they differ from one another in every size, constant and layer order."""
from __future__ import annotations

import os

from photon_infer_amd.config import SemezenConfig
from photon_infer_amd.weights import write_random_model


def _attn(heads, kv_heads, dim, scale, window=None, rot=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "scale": scale}
    if window is not None:
        m["mask"] = {"size": window}
    if rot is not None:
        m["rot"] = rot
    return m


def _rot(dims, base, factor=None, low=1.0, high=4.0, original=64):
    r = {"dims": dims, "base": base}
    if factor is not None:
        r["scaling"] = {"factor": factor, "low": low, "high": high, "original": original}
    return r


def _layer(kind, mixer, mlp):
    return {"type": kind, "mixer": mixer, "mlp": mlp}


def _gru(width):
    return {"width": width}


def _dense(ff):
    return {"kind": "dense", "ff": ff}


def _moe(ff, limit, experts, top):
    return {"kind": "moe", "expert": {"ff": ff, "limit": limit}, "router": {"experts": experts, "top": top}}


# A: two streams; windows of 7 and 20 under pages of 16; half a head rotated, short waves kept, long ones slowed by three, the rest
# blended; two of five experts, whose units are clamped early; both mixers under both kinds of feed-forward
TINY_A = {"architecture": "Semezen", "vocab": 300, "width": 64, "streams": 2, "norm": {"eps": 1e-6},
          "layers": [_layer("mingru", _gru(48), _dense(96)), _layer("attention", _attn(4, 2, 16, 0.3, 7, _rot(8, 100.0, 3.0)), _moe(40, 0.5, 5, 2)),
                     _layer("mingru", _gru(80), _moe(48, 0.8, 6, 3)), _layer("attention", _attn(2, 2, 32, 0.2, 20, _rot(16, 50.0, 2.0, 0.5, 2.0, 40)), _dense(72))]}

# B: sizes the matrix-core kernels take, four streams: heads of 64 and 32, one kv head under four, a whole head rotated, windows of
# 33 and 100, expert widths that are multiples of 32, attention first
TINY_B = {"architecture": "Semezen", "vocab": 776, "width": 256, "streams": 4, "norm": {"eps": 1e-5},
          "layers": [_layer("attention", _attn(4, 1, 64, 0.1, 33, _rot(64, 10000.0)), _moe(128, 1.5, 8, 4)), _layer("mingru", _gru(256), _dense(512)),
                     _layer("attention", _attn(8, 2, 32, 0.15, 100, _rot(16, 500.0, 4.0, 1.0, 8.0, 256)), _dense(320)),
                     _layer("mingru", _gru(192), _moe(96, 0.7, 7, 2))]}

# C: sizes that fit no fast kernel: a width that is no multiple of 4, an odd vocabulary, five streams, head sizes that are no
# multiples of 16 or 4, three kv heads, three rotated pairs, a layer that sees everything, one expert of nine, a layer
# without feed-forward after each mixer, pages of 8
TINY_C = {"architecture": "Semezen", "vocab": 257, "width": 90, "streams": 5, "norm": {"eps": 2e-6},
          "layers": [_layer("attention", _attn(6, 3, 12, 0.4, 5, _rot(6, 30.0, 8.0, 1.0, 4.0, 100)), None), _layer("mingru", _gru(37), _moe(36, 0.6, 9, 1)),
                     _layer("attention", _attn(3, 1, 10, 0.35, None, _rot(4, 20.0)), _dense(52)), _layer("mingru", _gru(70), None)]}

# D: one stream, one head, a window of one position, no rotation, an eps that counts, one expert alone and all of three
TINY_D = {"architecture": "Semezen", "vocab": 512, "width": 128, "streams": 1, "norm": {"eps": 0.05},
          "layers": [_layer("attention", _attn(1, 1, 48, 0.15, 1), _moe(48, 0.3, 1, 1)), _layer("attention", _attn(1, 1, 80, 0.12, 64, _rot(80, 200.0, 1.0)), None),
                     _layer("mingru", _gru(128), _moe(32, 2.0, 3, 3))]}

# E: recurrent layers only (no pages at all), nine streams
TINY_E = {"architecture": "Semezen", "vocab": 200, "width": 72, "streams": 9, "norm": {"eps": 1e-4},
          "layers": [_layer("mingru", _gru(72), None), _layer("mingru", _gru(20), _dense(40))]}

ALL = {"A": (TINY_A, dict(std=0.15, block_size=16, shut=3.0)), "B": (TINY_B, dict(std=0.08, block_size=16, shut=0.0)),
       "C": (TINY_C, dict(std=0.12, block_size=8, shut=2.0)), "D": (TINY_D, dict(std=0.1, block_size=16, shut=5.0)),
       "E": (TINY_E, dict(std=0.12, block_size=16, shut=4.0))}


def make_model_dir(tmp_path, name: str, seed: int = 0) -> str:
    """A model folder with random weights; ``shut`` is taken off the recurrences' gate biases (gates that are nearly shut
    make memories that reach far back)."""
    from safetensors.torch import load_file, save_file
    raw, init = ALL[name]
    d = os.path.join(str(tmp_path), f"semezen_{name}_{seed}")
    write_random_model(SemezenConfig.from_dict(raw), d, seed=seed, std=init["std"], norm_init="uniform", dtype="bfloat16")
    path = os.path.join(d, "model.safetensors")
    tensors = load_file(path)
    for n in tensors:
        if n.endswith("mix.z.b"):
            tensors[n] = tensors[n] - init["shut"]
    save_file(tensors, path)
    return d
