"""Typed configuration of the Fumanex decoder, read from its config.json.

A Fumanex model is a list of parallel layers: one RMS norm whose rows both the mixer and the
feed-forward read, their outputs added to the stream together.  The mixer is one of three: causal
grouped-query attention (biases; unit norms on q and k a head; no rotation, a learned bias by
bucket of distance instead; a score cap; a sliding window behind which the first positions stay
in sight; a learned sink a head; values mixed with those of the first layer that mixes), or one of
two linear attentions whose memory is a matrix a head with a fixed decay (retention: rotated q
and k, a unit norm and a silu gate a head; lightning: silu on q, k and v, one norm over all heads,
a sigmoid gate).  The feed-forward is two biased matrices around the tanh form of gelu.  Every
size and every constant that can differ between models comes from config.json; the layers may
all differ.

    {"architecture": "Fumanex", "vocab": V, "width": W, "norm": {"eps": e},
     "embedding": {"scale": c}, "logit_scale": s,
     "layers": [
       {"type": "attention",
        "mixer": {"heads": H, "kv_heads": G, "dim": d, "vdim": dv, "scale": s, "softcap": t,
                  "bias_max": D, "mask": {"size": w, "keep_first": f}, "v_mix": true}, "mlp": ...},
       {"type": "retention",
        "mixer": {"heads": H, "dim": d, "vdim": dv, "decay": [..H..],
                  "rot": {"dims": r, "base": b}}, "mlp": ...},
       {"type": "lightning",
        "mixer": {"heads": H, "dim": d, "vdim": dv, "decay": [..H..]}, "mlp": ...}]}
    mlp: null | {"kind": "dense", "ff": f}

Tensor names: ``embed``, ``head``, ``final.norm``, and per layer i under ``l<i>.``: ``norm1``; the
mixer's under ``mix.``: ``q q.b k k.b v v.b o o.b rel sink vmix`` (attention; ``rel`` [buckets,
heads] decides the number of buckets), ``q k v g o`` (retention), ``q k v g norm o`` (lightning);
the feed-forward's under ``mlp.``: ``up up.b down down.b``.
"""
from __future__ import annotations

import copy
from dataclasses import dataclass
from typing import Optional, Tuple

from ..errors import ConfigError
from .nupovik import _int, _num, _obj
from .registry import register_architecture
from .rotary import leading_rotary
from .specs import (DenseMlpSpec, DistanceBiasSpec, FixedDecayAttentionSpec, LeadingRotarySpec,
                    MaskedGqaAttentionSpec, ModelSpec, ParallelBlockSpec, RmsNormSpec,
                    ScheduleEntry)

# positions are 32-bit numbers in the kernels, and exact as such up to here
MAX_POSITIONS = 1 << 24
FF_ACTIVATION = "gelu_tanh"             # the design fixes it
MIXERS = ("attention", "retention", "lightning")


def _flag(d: dict, key: str, where: str) -> bool:
    v = d.get(key)
    if v is not None and not isinstance(v, bool):
        raise ConfigError(f"config.json: {where}{key!r} must be true or false, got {v!r}")
    return bool(v)


def _decays(m: dict, heads: int, where: str) -> Tuple[float, ...]:
    v = m.get("decay")
    if not isinstance(v, list) or len(v) != heads or any(
            isinstance(x, bool) or not isinstance(x, (int, float)) or not 0.0 <= x <= 1.0
            for x in v):
        raise ConfigError(f"config.json: {where}'decay' must be a list of {heads} numbers between "
                          f"0 and 1, got {v!r}")
    return tuple(float(x) for x in v)


def _rotary(m: dict, dim: int, where: str) -> Optional[LeadingRotarySpec]:
    if m.get("rot") is None:
        return None
    r = _obj(m, "rot", where)
    dims, base = _int(r, "dims", where + "rot.", 0), _num(r, "base", where + "rot.")
    if dims == 0:
        return None
    if dims > dim or dims % 2 != 0:
        raise ConfigError(f"config.json: {where}rot.dims={dims} must be even and at most dim={dim}")
    return leading_rotary(base, dims)


@dataclass(frozen=True)
class FumanexConfig:
    vocab: int
    width: int
    norm_eps: float
    embedding_scale: float
    logit_scale: float
    layers: Tuple[object, ...]                 # one ParallelBlockSpec a layer
    raw: dict

    # ------------------------------------------------------------------ parsing
    @classmethod
    def from_dict(cls, raw: dict) -> "FumanexConfig":
        vocab = _int(raw, "vocab", "")
        width = _int(raw, "width", "")
        eps = _num(_obj(raw, "norm", ""), "eps", "norm.")
        if not eps >= 0.0:
            raise ConfigError(f"config.json: norm.eps={eps} must not be negative")
        emb = 1.0
        if raw.get("embedding") is not None and \
                _obj(raw, "embedding", "").get("scale") is not None:
            emb = _num(raw["embedding"], "scale", "embedding.")
        scale = 1.0 if raw.get("logit_scale") is None else _num(raw, "logit_scale", "")
        layers = raw.get("layers")
        if not isinstance(layers, list) or not layers:
            raise ConfigError("config.json: 'layers' must be a list with at least one layer")
        blocks, source = [], None              # source: kv heads x vdim of the first that mixes
        for i, L in enumerate(layers):
            block, source = cls._block(i, L, width, eps, source)
            blocks.append(block)
        return cls(vocab, width, eps, emb, scale, tuple(blocks), copy.deepcopy(raw))

    @staticmethod
    def _norm(width: int, eps: float) -> RmsNormSpec:
        return RmsNormSpec(width, eps, weight_name="")     # the gain's tensor is the prefix itself

    @staticmethod
    def _block(i: int, L, width: int, eps: float, source):
        where = f"layers[{i}]."
        if not isinstance(L, dict):
            raise ConfigError(f"config.json: layers[{i}] must be an object")
        kind = L.get("type")
        if kind not in MIXERS:
            raise ConfigError(f"config.json: {where}type={kind!r}: the mixers of this design "
                              f"are {', '.join(repr(m) for m in MIXERS)}")
        m = _obj(L, "mixer", where)
        mw = where + "mixer."
        heads, dim, vdim = (_int(m, n, mw) for n in ("heads", "dim", "vdim"))
        if kind == "attention":
            mixer, source = FumanexConfig._attention(m, mw, width, eps, heads, dim, vdim, source)
        elif kind == "retention":
            mixer = FixedDecayAttentionSpec(
                hidden_size=width, n_heads=heads, head_dim=dim, value_dim=vdim,
                decay=_decays(m, heads, mw), norm_eps=eps, rotary=_rotary(m, dim, mw),
                k_scale=dim ** -0.5, norm="head", gate="silu")
        else:
            mixer = FixedDecayAttentionSpec(
                hidden_size=width, n_heads=heads, head_dim=dim, value_dim=vdim,
                decay=_decays(m, heads, mw), norm_eps=eps, silu=True, norm="row",
                norm_name="norm", gate="sigmoid")
        ff = None
        f, fw = L.get("mlp"), where + "mlp."
        if f is not None:
            if not isinstance(f, dict) or f.get("kind") != "dense":
                raise ConfigError(f"config.json: {fw}kind: the feed-forward of this design is "
                                  f"'dense', got {f!r}")
            ff = DenseMlpSpec(width, _int(f, "ff", fw), FF_ACTIVATION, bias=True, up_name="up",
                              down_name="down")
        return ParallelBlockSpec(mixer=mixer, feed_forward=ff,
                                 mixer_norm=FumanexConfig._norm(width, eps), ff_norm=None,
                                 mixer_prefix="mix.", ff_prefix="mlp.",
                                 mixer_norm_prefix="norm1"), source

    @staticmethod
    def _attention(m: dict, mw: str, width: int, eps: float, heads: int, dim: int, vdim: int,
                   source):
        kv = _int(m, "kv_heads", mw)
        if heads % kv != 0:
            raise ConfigError(f"config.json: {mw}kv_heads={kv} does not divide heads={heads}")
        window, keep = None, 0
        if m.get("mask") is not None:
            mask = _obj(m, "mask", mw)
            if mask.get("size") is not None:
                window = _int(mask, "size", mw + "mask.")
            if mask.get("keep_first") is not None:
                keep = _int(mask, "keep_first", mw + "mask.", 0)
        cap = None
        if m.get("softcap") is not None:
            cap = _num(m, "softcap", mw)
            if not cap > 0.0:
                raise ConfigError(f"config.json: {mw}softcap={cap} must be positive")
        far = _num(m, "bias_max", mw)
        if not far > 0.0:
            raise ConfigError(f"config.json: {mw}bias_max={far} must be positive")
        mix = "idle"
        if _flag(m, "v_mix", mw):
            mix = "source" if source is None else "blend"
            if source is not None and source != (kv, vdim):
                raise ConfigError(f"config.json: {mw}v_mix: {kv} kv heads of {vdim} values do not "
                                  f"mix with the first such layer's {source[0]} of {source[1]}")
            source = (kv, vdim)
        return MaskedGqaAttentionSpec(
            hidden_size=width, n_heads=heads, n_kv_heads=kv, head_dim=dim, value_dim=vdim,
            scale=_num(m, "scale", mw), qk_unit_eps=eps, bias=True, output_bias=True, softcap=cap,
            window=window, keep_first=keep if window is not None else 0,
            distance_bias=DistanceBiasSpec(far, name="rel"), sink=True, value_mix=mix, q_name="q",
            k_name="k", v_name="v", o_name="o", sink_name="sink", value_mix_name="vmix"), source

    def to_dict(self) -> dict:
        return copy.deepcopy(self.raw)

    @property
    def vocab_size(self) -> int:
        return self.vocab

    @property
    def model_type(self) -> str:
        return "fumanex"

    # ------------------------------------------------------------------ the model's parts
    def model_spec(self) -> ModelSpec:
        return ModelSpec(
            vocab_size=self.vocab, hidden_size=self.width, max_positions=MAX_POSITIONS,
            layers=self.layers, schedule=tuple(ScheduleEntry(i) for i in range(len(self.layers))),
            final_norm=self._norm(self.width, self.norm_eps), tie_word_embeddings=False,
            embed_name="embed", final_norm_prefix="final.norm", head_name="head",
            layer_prefix="l{}.", embedding_multiplier=self.embedding_scale,
            logit_scale=self.logit_scale)


register_architecture("Fumanex", FumanexConfig)
