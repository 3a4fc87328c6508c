"""Typed configuration of the Tigesun decoder, read from its config.json.

A Tigesun model passes the embedding's rows through a norm and then runs a list of layers with an
RMS norm before and behind every sublayer.  The mixer is one of three: causal grouped-query
attention (a norm a head on q and k, some leading elements of a head rotated, the rotation's
frequencies stretched by turns), attention over one latent row a token (no positions, no query
latent, a sliding window), or a state space with one decay a head and token behind short
convolutions, gated and then normed in parts.  The feed-forward, which a layer may lack, is a gated
one (the tanh form of gelu) with biases.  The head is the embedding, its logits are capped.  A
layer may run with another layer's tensors and a cache and state of its own.  Every size and every
constant that can differ between models comes from config.json; the layers may all differ.

    {"architecture": "Tigesun", "vocab": V, "width": W, "norm": {"eps": e}, "logit_softcap": c,
     "layers": [
       {"type": "attention",
        "mixer": {"heads": H, "kv_heads": G, "dim": d, "vdim": dv, "scale": s,
                  "rot": {"dims": r, "base": b,
                          "scaling": {"factor", "original", "fast", "slow"}}}, "mlp": ...},
       {"type": "latent_attention",
        "mixer": {"heads": H, "dim": d, "vdim": dv, "kv_rank": k, "scale": s,
                  "mask": {"size": window}}, "mlp": ...},
       {"type": "mamba2",
        "mixer": {"heads": H, "vdim": dv, "state": N, "groups": G, "conv": taps,
                  "norm_groups": P}, "mlp": ...},
       {..., "weights_of": j}]}
    mlp: null | {"kind": "dense", "ff": f}

Tensor names: ``embed``, ``embed.norm``, ``final.norm``, and per layer i under ``l<i>.``: ``norm1
norm1b`` and (with a feed-forward) ``norm2 norm2b``; the mixer's under ``mix.``: ``q k v q.norm
k.norm o`` (attention), ``q dkv dkv.norm uk uv o`` (latent_attention), ``in conv conv.b dt_bias
A_log D norm o`` (mamba2); the feed-forward's under ``mlp.``: ``gate gate.b up up.b down down.b``.
"""
from __future__ import annotations

import copy
from dataclasses import dataclass
from typing import Optional, Tuple

from ..errors import ConfigError
from .kugisun import weight_owners
from .nupovik import _int, _num, _obj
from .registry import register_architecture
from .rotary import leading_rotary
from .specs import (GatedMlpSpec, LatentAttentionSpec, LayerNormSpec, LeadingRotarySpec,
                    MaskedGqaAttentionSpec, ModelSpec, SandwichNormBlockSpec, ScheduleEntry,
                    StateSpaceSpec)

# positions are 32-bit numbers in the kernels, and exact as such up to here
MAX_POSITIONS = 1 << 24
FF_ACTIVATION = "gelu_tanh"             # the design fixes it
MIXERS = ("attention", "latent_attention", "mamba2")


def _rotary(m: dict, dim: int, where: str) -> Optional[LeadingRotarySpec]:
    if m.get("rot") is None:
        return None
    r, rw = _obj(m, "rot", where), where + "rot."
    dims = _int(r, "dims", rw, 0)
    if dims == 0:
        return None
    if dims > dim or dims % 2 != 0:
        raise ConfigError(f"config.json: {rw}dims={dims} must be even and at most dim={dim}")
    scaling = r.get("scaling")
    if scaling is not None and not isinstance(scaling, dict):
        raise ConfigError(f"config.json: {rw}scaling must be an object or null")
    return leading_rotary(_num(r, "base", rw), dims, scaling)


@dataclass(frozen=True)
class TigesunConfig:
    vocab: int
    width: int
    norm_eps: float
    logit_softcap: Optional[float]
    layers: Tuple[object, ...]            # one SandwichNormBlockSpec for every layer with tensors
    layer_numbers: Tuple[int, ...]        # the number each of them goes by in the file
    order: Tuple[int, ...]                # for every run, the index into ``layers``
    raw: dict

    # ------------------------------------------------------------------ parsing
    @classmethod
    def from_dict(cls, raw: dict) -> "TigesunConfig":
        vocab = _int(raw, "vocab", "")
        width = _int(raw, "width", "")
        eps = _num(_obj(raw, "norm", ""), "eps", "norm.")
        if not eps >= 0.0:
            raise ConfigError(f"config.json: norm.eps={eps} must not be negative")
        cap = None if raw.get("logit_softcap") is None else _num(raw, "logit_softcap", "")
        if cap is not None and not cap > 0.0:
            raise ConfigError(f"config.json: logit_softcap={cap} must be positive")
        layers = raw.get("layers")
        if not isinstance(layers, list) or not layers:
            raise ConfigError("config.json: 'layers' must be a list with at least one layer")
        owners = weight_owners(layers)
        numbers = tuple(sorted(set(owners)))
        blocks = tuple(cls._block(j, layers[j], width, eps) for j in numbers)
        order = tuple(numbers.index(j) for j in owners)
        return cls(vocab, width, eps, cap, blocks, numbers, order, copy.deepcopy(raw))

    @staticmethod
    def _norm(width: int, eps: float) -> LayerNormSpec:
        # x / sqrt(mean x^2 + eps) * w: not centred, no bias; the gain's tensor is the prefix itself
        return LayerNormSpec(width, eps, centred=False, weight_name="", bias_name=None)

    @staticmethod
    def _block(i: int, L: dict, width: int, eps: float) -> SandwichNormBlockSpec:
        where = f"layers[{i}]."
        kind = L.get("type")
        make = {"attention": TigesunConfig._attention, "latent_attention": TigesunConfig._latent,
                "mamba2": TigesunConfig._state_space}.get(kind)
        if make is None:
            raise ConfigError(f"config.json: {where}type={kind!r}: the mixers of this design "
                              f"are {', '.join(repr(m) for m in MIXERS)}")
        mixer = make(_obj(L, "mixer", where), where + "mixer.", width, eps)
        norm, ff = TigesunConfig._norm(width, eps), None
        f, fw = L.get("mlp"), where + "mlp."
        if f is not None:
            if not isinstance(f, dict) or f.get("kind") != "dense":
                raise ConfigError(f"config.json: {fw}kind: the feed-forward of this design is "
                                  f"'dense', got {f!r}")
            ff = GatedMlpSpec(width, _int(f, "ff", fw), FF_ACTIVATION, bias=True, gate_name="gate",
                              up_name="up", down_name="down")
        return SandwichNormBlockSpec(
            mixer=mixer, feed_forward=ff, mixer_norm=norm, mixer_post_norm=norm,
            ff_norm=norm if ff is not None else None, ff_post_norm=norm if ff is not None else None,
            mixer_prefix="mix.", ff_prefix="mlp.", mixer_norm_prefix="norm1",
            mixer_post_norm_prefix="norm1b", ff_norm_prefix="norm2", ff_post_norm_prefix="norm2b")

    @staticmethod
    def _attention(m: dict, mw: str, width: int, eps: float) -> MaskedGqaAttentionSpec:
        heads, kv, dim = _int(m, "heads", mw), _int(m, "kv_heads", mw), _int(m, "dim", mw)
        if heads % kv != 0:
            raise ConfigError(f"config.json: {mw}heads={heads} is no multiple of kv_heads={kv}")
        return MaskedGqaAttentionSpec(
            hidden_size=width, n_heads=heads, n_kv_heads=kv, head_dim=dim,
            value_dim=_int(m, "vdim", mw), scale=_num(m, "scale", mw), qk_norm_eps=eps,
            qk_norm_per_head=True, rotary=_rotary(m, dim, mw), q_name="q", k_name="k", v_name="v",
            o_name="o", q_norm_name="q.norm", k_norm_name="k.norm")

    @staticmethod
    def _latent(m: dict, mw: str, width: int, eps: float) -> LatentAttentionSpec:
        window = None
        if m.get("mask") is not None:
            window = _int(_obj(m, "mask", mw), "size", mw + "mask.")
        return LatentAttentionSpec(
            hidden_size=width, n_heads=_int(m, "heads", mw), head_dim=_int(m, "dim", mw), rot_dim=0,
            value_dim=_int(m, "vdim", mw), q_rank=None, kv_rank=_int(m, "kv_rank", mw),
            scale=_num(m, "scale", mw), norm_eps=eps, window=window, uq_name="q", dkv_name="dkv",
            dkv_norm_name="dkv.norm", uk_name="uk", uv_name="uv", o_name="o")

    @staticmethod
    def _state_space(m: dict, mw: str, width: int, eps: float) -> StateSpaceSpec:
        heads, vdim = _int(m, "heads", mw), _int(m, "vdim", mw)
        groups, parts = _int(m, "groups", mw), _int(m, "norm_groups", mw)
        if heads % groups != 0:
            raise ConfigError(f"config.json: {mw}heads={heads} is no multiple of groups={groups}")
        if heads * vdim % parts != 0:
            raise ConfigError(f"config.json: {mw}norm_groups={parts} does not divide the heads' "
                              f"{heads * vdim} values")
        return StateSpaceSpec(
            hidden_size=width, n_heads=heads, value_dim=vdim, state_dim=_int(m, "state", mw),
            n_groups=groups, conv_taps=_int(m, "conv", mw), norm_groups=parts, norm_eps=eps)

    def to_dict(self) -> dict:
        return copy.deepcopy(self.raw)

    @property
    def vocab_size(self) -> int:
        return self.vocab

    @property
    def model_type(self) -> str:
        return "tigesun"

    # ------------------------------------------------------------------ the model's parts
    def model_spec(self) -> ModelSpec:
        """Every run of a layer, also one with another layer's tensors, has a cache and a state
        of its own."""
        norm = self._norm(self.width, self.norm_eps)
        return ModelSpec(
            vocab_size=self.vocab, hidden_size=self.width, max_positions=MAX_POSITIONS,
            layers=self.layers, schedule=tuple(ScheduleEntry(i) for i in self.order),
            final_norm=norm, tie_word_embeddings=True, embed_name="embed",
            final_norm_prefix="final.norm", head_name="head", layer_prefix="l{}.",
            embedding_norm=norm, embedding_norm_prefix="embed.norm",
            logit_softcap=self.logit_softcap, layer_numbers=self.layer_numbers)


register_architecture("Tigesun", TigesunConfig)
