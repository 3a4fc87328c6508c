"""Small Fumanex configurations for the tests, and weights made for them.  They differ from each
other in every size and option: the mixers in every order, layers without a feed-forward, values
mixed or not (also with layers between that do not mix), windows of one token, under a page,
several pages and none, kept first positions from none to more than a page and more than the
window, one kv head and kv heads = heads, values narrower and wider than keys, buckets of
distances from two to thirty-two, rotations of a part of a head, of the whole head and none,
decays of 0, 1 and between, heads of one element, caps and none; widths that no vector kernel
takes and widths the bfloat16 matrix and MFMA kernels take."""
from __future__ import annotations

from typing import Dict

import torch

from zinfer_amd.config import FumanexConfig
from zinfer_amd.models.build import declare_tensors


def _dense(ff):
    return None if ff is None else {"kind": "dense", "ff": ff}


def _attention(heads, kv, dim, vdim, ff, size, keep, far, cap=5.0, mix=True, scale=None):
    m = {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim,
         "scale": scale if scale is not None else 1.7 / dim ** 0.5, "softcap": cap,
         "bias_max": far, "v_mix": mix,
         "mask": None if size is None else {"size": size, "keep_first": keep}}
    return {"type": "attention", "mixer": m, "mlp": _dense(ff)}


def _retention(heads, dim, vdim, ff, dims, base, decay):
    m = {"heads": heads, "dim": dim, "vdim": vdim, "decay": decay,
         "rot": None if dims is None else {"dims": dims, "base": base}}
    return {"type": "retention", "mixer": m, "mlp": _dense(ff)}


def _lightning(heads, dim, vdim, ff, decay):
    return {"type": "lightning", "mixer": {"heads": heads, "dim": dim, "vdim": vdim,
                                           "decay": decay}, "mlp": _dense(ff)}


# all three mixers; a layer that does not mix its values between two that do; layers without
# a feed-forward; a window of 9 with 3 kept positions and one of 5 with none
FX_A = {"architecture": "Fumanex", "vocab": 203, "width": 48, "norm": {"eps": 1e-5},
        "embedding": {"scale": 3.5}, "logit_scale": 0.6,
        "layers": [_attention(6, 3, 12, 20, 40, 9, 3, 40),
                   _retention(3, 20, 12, 36, 12, 500.0, [0.9, 1.0, 0.5]),
                   _attention(4, 1, 16, 8, None, 30, 18, 25.5, mix=False),
                   _lightning(2, 6, 10, 24, [0.75, 0.99]),
                   _attention(3, 3, 8, 20, 52, 5, 0, 17, cap=2.0),
                   _retention(1, 8, 30, None, 8, 10000.0, [0.97])]}

# a lightning layer first; a window of one token with one kept position; kv heads = heads;
# decays of 0 and 1; no logit scale; the widest kept range beyond a page of 8
FX_B = {"architecture": "Fumanex", "vocab": 310, "width": 72, "norm": {"eps": 1e-6},
        "embedding": {"scale": 8.0},
        "layers": [_lightning(3, 12, 16, 44, [0.0, 1.0, 0.8]),
                   _attention(5, 5, 8, 12, 24, 1, 1, 9.0),
                   _attention(10, 5, 24, 12, 32, 20, 11, 300, cap=8.0),
                   _retention(4, 4, 8, 20, 2, 50.0, [0.99, 0.9, 0.6, 1.0]),
                   _lightning(1, 40, 4, None, [0.95]),
                   _attention(5, 5, 16, 12, 64, None, 0, 70, cap=None)]}

# a width no vector kernel takes, sizes that are no multiple of 4; kept positions beyond the
# window; heads of one element; a retention without a rotation
FX_C = {"architecture": "Fumanex", "vocab": 97, "width": 50, "norm": {"eps": 1e-3},
        "embedding": {"scale": 1.0}, "logit_scale": 2.5,
        "layers": [_retention(5, 7, 3, 14, None, 1.0, [0.3, 0.6, 0.9, 0.95, 1.0]),
                   _attention(5, 1, 7, 5, 30, 7, 22, 12.0),
                   _lightning(7, 1, 1, 10, [0.9] * 7),
                   _attention(3, 1, 10, 5, 18, 17, 2, 33.0, cap=1.5),
                   _retention(2, 10, 11, 22, 6, 7.0, [0.98, 0.85])]}

# widths the bfloat16 matrix kernels take, head sizes of the MFMA attention and of the chunked
# recurrence; a window under a chunk of 128 tokens
FX_D = {"architecture": "Fumanex", "vocab": 512, "width": 128, "norm": {"eps": 1e-6},
        "embedding": {"scale": 11.0}, "logit_scale": 1.5,
        "layers": [_attention(6, 2, 64, 32, 192, 70, 5, 64.0, cap=20.0),
                   _retention(2, 64, 96, 128, 32, 10000.0, [0.99, 0.999]),
                   _lightning(4, 32, 64, 64, [0.6, 0.9, 0.97, 0.998]),
                   _attention(4, 2, 32, 32, 128, 33, 40, 200.0, cap=10.0),
                   _retention(1, 128, 160, 64, 128, 100000.0, [0.995]),
                   _lightning(2, 96, 24, 96, [0.95, 0.9995])]}

CONFIGS = {"A": FX_A, "B": FX_B, "C": FX_C, "D": FX_D}
PAGE_SIZE = {"A": 16, "B": 8, "C": 4, "D": 16}
BUCKETS = {"A": (8, 12, 6), "B": (4, 32, 10), "C": (6, 16), "D": (32, 8)}


def config_of(name: str) -> FumanexConfig:
    return FumanexConfig.from_dict(CONFIGS[name])


def weights_of(name: str, seed: int = 0, dtype=torch.float32) -> Dict[str, torch.Tensor]:
    """Weights large enough that every mechanism shows: gains around 1, biases and sinks of the
    scores' size, biases by distance that differ from bucket to bucket, shares of the first
    values between a third and two thirds.  Values are rounded to bfloat16 (and stored as
    ``dtype``), so that both compute dtypes see the same."""
    cfg = config_of(name)
    decls = declare_tensors(cfg.model_spec())
    g = torch.Generator().manual_seed(4000 + seed)
    out = {}
    tables = iter(BUCKETS[name])
    for n, d in decls.items():
        shape = d.drawn_shape()
        last = n.split(".")[-1]
        if last == "rel":
            shape = (next(tables), shape[1])
        if "norm" in n:
            t = 1.0 + 0.3 * torch.randn(shape, generator=g)
        elif last == "vmix":
            t = 0.3 + 0.4 * torch.rand(shape, generator=g)
        elif last == "sink":
            t = 1.5 * torch.randn(shape, generator=g)
        elif last == "rel":
            t = 1.2 * torch.randn(shape, generator=g)
        elif last == "b":
            t = 0.5 * torch.randn(shape, generator=g)
        elif n == "embed":
            t = torch.randn(shape, generator=g) / CONFIGS[name]["embedding"]["scale"]
        else:
            t = torch.randn(shape, generator=g) * (1.5 / shape[-1] ** 0.5)
        out[n] = t.to(torch.bfloat16).to(dtype)
    return out


def tokens(n: int, vocab: int, seed: int):
    g = torch.Generator().manual_seed(seed)
    return torch.randint(0, vocab, (n,), generator=g).tolist()
