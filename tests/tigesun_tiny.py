"""Small Tigesun configurations for the tests, and weights made for them.  They differ from each
other in every size and option: the mixers in every order, layers with and without a feed-forward
of every kind, layers that run with another layer's tensors (also through a second such layer, and
of a layer that comes later), one kv head and kv heads = heads, values narrower and wider than
keys, rotations of a part of a head, of the whole head and none, stretched or not, windows of one
token, under a page, several pages and none, latents narrower and wider than a head, one to five
taps, one group and a group a head, one head, heads of one value, states that are no multiple of 4,
one norm over all heads and parts that cut through heads, a cap and none; widths that no vector
kernel takes and widths the bfloat16 matrix and MFMA kernels take."""
from __future__ import annotations

from typing import Dict

import torch

from zinfer_amd.config import TigesunConfig
from zinfer_amd.models.build import declare_tensors


def _dense(ff):
    return None if ff is None else {"kind": "dense", "ff": ff}


def _attention(heads, kv, dim, vdim, ff, dims=None, base=500.0, scaling=None):
    rot = None if dims is None else {"dims": dims, "base": base}
    if scaling is not None:
        rot["scaling"] = dict(zip(("factor", "original", "fast", "slow"), scaling))
    return {"type": "attention", "mlp": _dense(ff),
            "mixer": {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim,
                      "scale": 1.3 / dim ** 0.5, "rot": rot}}


def _latent(heads, dim, vdim, rank, ff, size):
    return {"type": "latent_attention", "mlp": _dense(ff),
            "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "kv_rank": rank,
                      "scale": 1.6 / dim ** 0.5, "mask": None if size is None else {"size": size}}}


def _space(heads, vdim, state, groups, conv, parts, ff=None):
    return {"type": "mamba2", "mlp": _dense(ff),
            "mixer": {"heads": heads, "vdim": vdim, "state": state, "groups": groups, "conv": conv,
                      "norm_groups": parts}}


def _again(layers, j):
    """The entry of a layer that runs with layer j's tensors."""
    return dict(layers[j], weights_of=j)


# every mixer; a state space without a feed-forward and one with it; the first three run again
_A = [_attention(6, 3, 12, 20, 40, 8, 100.0, (3.0, 40, 4.0, 0.5)), _space(3, 16, 10, 1, 4, 3),
      _latent(4, 10, 12, 18, 36, 9), _space(4, 6, 12, 2, 2, 1, 28), _latent(2, 16, 5, 24, None, 30)]
TG_A = {"architecture": "Tigesun", "vocab": 203, "width": 48, "norm": {"eps": 1e-5},
        "logit_softcap": 25.0,
        "layers": _A + [_again(_A, 0), _again(_A, 1), _again(_A, 2)]}

# a state space first, tensors of a layer that comes later, and a chain of such layers; no cap; a
# window of one token and none; rotations whole and not at all; one tap; norm parts of a head and a half
_B = [_space(6, 4, 8, 6, 1, 4, 24), _attention(5, 5, 8, 12, 24, 8, 50.0), _latent(3, 8, 16, 20, 44, 1),
      _attention(10, 5, 24, 12, 32), _latent(5, 24, 8, 16, None, None), _space(4, 16, 40, 1, 5, 2)]
TG_B = {"architecture": "Tigesun", "vocab": 310, "width": 72, "norm": {"eps": 1e-6},
        "layers": [dict(_B[5], weights_of=6)] + _B + [dict(_B[1], weights_of=2),
                                                      dict(_B[1], weights_of=7)]}

# a width no vector kernel takes, sizes that are no multiple of 4, one head, one kv head, heads of
# one value
_C = [_latent(1, 7, 3, 5, 14, 7), _space(5, 3, 7, 5, 3, 1), _attention(5, 1, 10, 5, 30, 6, 7.0),
      _space(7, 1, 1, 1, 4, 1, 18), _attention(3, 1, 6, 11, None, 2, 20.0, (2.5, 100, 8.0, 2.0)),
      _space(1, 12, 30, 1, 2, 2)]
TG_C = {"architecture": "Tigesun", "vocab": 97, "width": 50, "norm": {"eps": 1e-3},
        "logit_softcap": 12.0, "layers": _C + [_again(_C, 1), _again(_C, 4)]}

# widths the bfloat16 matrix kernels take, sizes of the MFMA attention and of the recurrence in
# chunks (one, two and four heads a group; values of one block, of two, and of less than one)
_D = [_attention(4, 2, 64, 64, 192, 64, 10000.0, (4.0, 256, 32.0, 1.0)), _space(8, 32, 64, 2, 4, 2),
      _latent(6, 32, 64, 64, 128, 70), _space(4, 96, 128, 1, 3, 4, 64), _attention(6, 6, 32, 96, 96, 16),
      _space(3, 64, 24, 3, 2, 1)]
TG_D = {"architecture": "Tigesun", "vocab": 512, "width": 128, "norm": {"eps": 1e-6},
        "logit_softcap": 30.0, "layers": _D + [_again(_D, 1), _again(_D, 2)]}

CONFIGS = {"A": TG_A, "B": TG_B, "C": TG_C, "D": TG_D}
PAGE_SIZE = {"A": 16, "B": 8, "C": 4, "D": 16}


def config_of(name: str) -> TigesunConfig:
    return TigesunConfig.from_dict(CONFIGS[name])


def weights_for(raw: dict, seed: int = 0, dtype=torch.float32) -> Dict[str, torch.Tensor]:
    """Weights large enough that every mechanism shows: gains around 1, biases of the rows' size,
    taps of like size, decays from nearly none to more than half a token, step sizes from a
    hundredth to one.  Values are rounded to bfloat16 (and stored as ``dtype``), so that both
    compute dtypes see the same."""
    decls = declare_tensors(TigesunConfig.from_dict(raw).model_spec())
    g = torch.Generator().manual_seed(6000 + seed)
    out = {}
    for n, d in decls.items():
        if n == "head":
            continue                                  # the embedding
        shape, last = d.drawn_shape(), n.split(".")[-1]
        if "norm" in n:
            t = 1.0 + 0.3 * torch.randn(shape, generator=g)
        elif last == "conv":
            t = torch.randn(shape, generator=g) * (0.9 / shape[1] ** 0.5)
        elif last == "A_log":
            t = -4.0 + 4.5 * torch.rand(shape, generator=g)
        elif last == "dt_bias":
            t = -3.0 + 2.5 * torch.rand(shape, generator=g)
        elif last == "D":
            t = torch.randn(shape, generator=g)
        elif last == "b":
            t = 0.5 * torch.randn(shape, generator=g)
        elif n == "embed":
            t = torch.randn(shape, generator=g)
        else:
            t = torch.randn(shape, generator=g) * (1.5 / shape[-1] ** 0.5)
        out[n] = t.to(torch.bfloat16).to(dtype)
    return out


def weights_of(name: str, seed: int = 0, dtype=torch.float32) -> Dict[str, torch.Tensor]:
    return weights_for(CONFIGS[name], seed, dtype)


def tokens(n: int, vocab: int, seed: int):
    g = torch.Generator().manual_seed(seed)
    return torch.randint(0, vocab, (n,), generator=g).tolist()
