"""Tiny Roserax configurations for tests; they differ from one another in every size, constant and layer order."""
from __future__ import annotations

import os

from photon_infer_amd.config import RoseraxConfig
from photon_infer_amd.weights import write_random_model


def _layer(kind, mixer, mlp):
    return {"type": kind, "mixer": mixer, "mlp": mlp}


def _attn(heads, kv_heads, dim, vdim, scale, size=None, keep=0):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale}
    if size is not None:
        m["mask"] = {"size": size, "keep_first": keep}
    return m


def _latent(heads, dim, rot_dim, vdim, q_rank, kv_rank, scale, base):
    return {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "q_rank": q_rank, "kv_rank": kv_rank, "scale": scale,
            "rot": {"base": base, "dims": rot_dim}}


def _ret(dim, vdim, decay, base, dims):
    return {"heads": len(decay), "dim": dim, "vdim": vdim, "decay": list(decay), "rot": {"base": base, "dims": dims}}


def _dense(ff):
    return {"kind": "dense", "ff": ff}


def _moe(ff, experts, top, count=None, keep=None):
    r = {"experts": experts, "top": top}
    if count is not None:
        r["groups"] = {"count": count, "keep": keep}
    return {"kind": "moe", "expert": {"ff": ff}, "router": r}


def _model(vocab, width, emb, logit, eps, layers):
    return {"architecture": "Roserax", "vocab": vocab, "width": width, "embedding": {"scale": emb}, "logit_scale": logit, "norm": {"eps": eps},
            "layers": layers}


# A: a window that is no multiple of the page and keeps part of a page; a second one that keeps more than a page; values of another
# width than keys; all kinds of mixer, all kinds of feed-forward and none; two of six experts in three groups, two of them kept
TINY_A = _model(300, 64, 4.0, 0.7, 1e-6, [
    _layer("attention", _attn(4, 2, 16, 16, 0.35, 21, 5), _moe(48, 6, 2, 3, 2)), _layer("retention", _ret(16, 24, [0.9, 0.99, 1.0], 500.0, 16), _dense(80)),
    _layer("latent_attention", _latent(2, 16, 8, 24, 20, 24, 0.3, 300.0), _moe(40, 5, 3)), _layer("attention", _attn(2, 1, 24, 16, 0.3, 40, 19), None),
    _layer("retention", _ret(8, 16, [0.5, 0.97], 40.0, 4), None)])

# B: sizes the matrix-core kernels take; the kept tokens fill more than a chunk of 32 keys; a layer that sees everything; one
# group of three kept; heads of 64 on one kv head
TINY_B = _model(776, 192, 8.0, 0.5, 1e-5, [
    _layer("latent_attention", _latent(4, 32, 16, 32, 64, 48, 0.15, 10000.0), _dense(512)), _layer("attention", _attn(4, 1, 64, 64, 0.12, 50, 37), _moe(64, 9, 2, 3, 1)),
    _layer("retention", _ret(32, 64, [0.96875, 0.999], 10000.0, 32), _moe(128, 4, 4)), _layer("attention", _attn(6, 2, 32, 32, 0.2), _dense(256)),
    _layer("attention", _attn(4, 2, 48, 48, 0.15, 100, 1), _dense(128))])

# C: sizes that fit no fast kernel: a width that is no multiple of 4, an odd vocabulary, head sizes that are no multiples of 16 or
# 4, three kv heads, more kept tokens than the window holds, a window shorter than a page, rotations of a part, pages of 8
TINY_C = _model(257, 90, 1.0, 1.0, 2e-6, [
    _layer("retention", _ret(10, 7, [0.98, 0.8, 0.0], 30.0, 6), None), _layer("attention", _attn(6, 3, 12, 10, 0.4, 5, 11), _dense(52)),
    _layer("latent_attention", _latent(3, 10, 6, 14, 11, 30, 0.3, 50.0), None), _layer("attention", _attn(3, 1, 9, 9, 0.35, 13, 0), _moe(36, 7, 1)),
    _layer("retention", _ret(6, 9, [0.995], 100.0, 2), _moe(20, 4, 2, 4, 2))])

# D: one head everywhere, a window of one position with one kept token, a latent row wider than 256, an eps that counts, one
# expert alone
TINY_D = _model(512, 128, 11.3, 2.5, 0.02, [
    _layer("attention", _attn(1, 1, 80, 48, 0.15, 1, 1), _moe(48, 1, 1)), _layer("latent_attention", _latent(1, 24, 16, 40, 32, 272, 0.12, 1000.0), _dense(96)),
    _layer("retention", _ret(48, 80, [0.9999], 200.0, 40), _dense(160))])

# E: retention only (no pages at all)
TINY_E = _model(200, 72, 2.0, 0.25, 1e-4, [_layer("retention", _ret(20, 36, [0.7, 0.95], 90.0, 12), None),
                                           _layer("retention", _ret(36, 20, [0.99, 0.3, 0.999, 0.9], 1000.0, 36), _dense(40))])

ALL = {"A": (TINY_A, dict(std=0.2, block_size=16)), "B": (TINY_B, dict(std=0.1, block_size=16)), "C": (TINY_C, dict(std=0.2, block_size=8)),
       "D": (TINY_D, dict(std=0.12, block_size=16)), "E": (TINY_E, dict(std=0.15, block_size=16))}


def make_model_dir(tmp_path, name: str, seed: int = 0) -> str:
    """A model folder with random weights."""
    raw, init = ALL[name]
    d = os.path.join(str(tmp_path), f"roserax_{name}_{seed}")
    return write_random_model(RoseraxConfig.from_dict(raw), d, seed=seed, std=init["std"], norm_init="uniform", dtype="bfloat16")
