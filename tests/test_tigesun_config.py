"""The Tigesun configuration on the CPU: what config.json gives, whose tensors a layer runs with,
what is refused, the cache or state each run asks for, the tensors a model declares, how the
recurrence's heads are dealt, a model folder written and read, and the plain implementation's own
pieces by hand."""
import copy
import json
import math
import os

import pytest
import torch

import plain_tigesun as P
import tigesun_tiny as tt
from zinfer_amd import ops
from zinfer_amd.config import (GatedMlpSpec, LatentAttentionSpec, LayerNormSpec,
                               MaskedGqaAttentionSpec, SandwichNormBlockSpec, StateSpaceSpec,
                               TigesunConfig, entry_for)
from zinfer_amd.errors import ConfigError
from zinfer_amd.models.build import declare_tensors
from zinfer_amd.models.decoder import DecoderModel
from zinfer_amd.parts.base import BuildContext, KVNeed, StateNeed


def test_registry_finds_the_family_by_its_one_name():
    assert entry_for(tt.TG_A).config_type is TigesunConfig
    assert entry_for({"architecture": "Tigesun", "model_type": "qwen3"}).config_type is TigesunConfig


@pytest.mark.parametrize("name", sorted(tt.CONFIGS))
def test_sizes_and_constants_come_from_the_file(name):
    raw = tt.CONFIGS[name]
    spec = tt.config_of(name).model_spec()
    W, eps = raw["width"], raw["norm"]["eps"]
    norm = LayerNormSpec(W, eps, centred=False, weight_name="", bias_name=None)
    assert (spec.vocab_size, spec.hidden_size) == (raw["vocab"], W)
    assert spec.tie_word_embeddings and spec.logit_softcap == raw.get("logit_softcap")
    assert spec.embedding_norm == norm == spec.final_norm
    assert spec.embedding_norm_prefix == "embed.norm" and spec.embedding_multiplier == 1.0
    assert len(spec.schedule) == len(raw["layers"])
    assert all(e.cache_of is None for e in spec.schedule)
    for i, (L, e) in enumerate(zip(raw["layers"], spec.schedule)):
        assert spec.layer_numbers[e.layer] == P.owner(raw, i)
        block, r = spec.layers[e.layer], L["mixer"]
        assert isinstance(block, SandwichNormBlockSpec)
        assert block.mixer_norm == block.mixer_post_norm == norm
        m = block.mixer
        if L["type"] == "attention":
            assert isinstance(m, MaskedGqaAttentionSpec)
            assert (m.n_heads, m.n_kv_heads, m.head_dim, m.value_dim, m.scale, m.qk_norm_eps) == \
                (r["heads"], r["kv_heads"], r["dim"], r["vdim"], r["scale"], eps)
            assert m.qk_norm_per_head and not (m.bias or m.sink or m.head_gate)
            assert m.window is m.chunk is m.softcap is None
            if r["rot"] is None:
                assert m.rotary is None
            else:
                freqs, length = P.stretched(r["rot"]["base"], r["rot"]["dims"], r["rot"].get("scaling"))
                assert m.rotary.dims == r["rot"]["dims"] and not m.rotary.interleaved
                assert m.rotary.magnitude == pytest.approx(length, rel=1e-12)
                assert m.rotary.frequencies == pytest.approx(freqs, rel=1e-12)
        elif L["type"] == "latent_attention":
            assert isinstance(m, LatentAttentionSpec)
            assert (m.n_heads, m.head_dim, m.value_dim, m.kv_rank, m.scale, m.norm_eps) == \
                (r["heads"], r["dim"], r["vdim"], r["kv_rank"], r["scale"], eps)
            assert m.rot_dim == 0 and m.q_rank is None and m.rotary is None
            assert m.window == (r["mask"] or {"size": None})["size"] and m.chunk is None
        else:
            assert m == StateSpaceSpec(W, r["heads"], r["vdim"], r["state"], r["groups"], r["conv"],
                                       r["norm_groups"], eps)
        f = block.feed_forward
        if L["mlp"] is None:
            assert f is None and block.ff_norm is None and block.ff_post_norm is None
        else:
            assert f == GatedMlpSpec(W, L["mlp"]["ff"], "gelu_tanh", True, gate_name="gate",
                                     up_name="up", down_name="down")
            assert block.ff_norm == block.ff_post_norm == norm


def test_what_the_configuration_refuses():
    def broken(change, base=tt.TG_A):
        raw = copy.deepcopy(base)
        change(raw)
        with pytest.raises(ConfigError):
            TigesunConfig.from_dict(raw)
    broken(lambda r: r.pop("vocab"))
    broken(lambda r: r.update(width=0))
    broken(lambda r: r["norm"].update(eps=-1.0))
    broken(lambda r: r.pop("norm"))
    broken(lambda r: r.update(logit_softcap=0.0))
    broken(lambda r: r.update(layers=[]))
    broken(lambda r: r["layers"].append(7))
    broken(lambda r: r["layers"][0].update(type="retention"))
    broken(lambda r: r["layers"][0].pop("mixer"))
    broken(lambda r: r["layers"][0]["mixer"].update(kv_heads=4))            # of 6 heads
    broken(lambda r: r["layers"][0]["mixer"].pop("scale"))
    broken(lambda r: r["layers"][0]["mixer"]["rot"].update(dims=5))
    broken(lambda r: r["layers"][0]["mixer"]["rot"].update(dims=14))        # heads of 12
    broken(lambda r: r["layers"][0]["mixer"]["rot"].pop("base"))
    broken(lambda r: r["layers"][0]["mixer"]["rot"]["scaling"].pop("slow"))
    broken(lambda r: r["layers"][0]["mixer"]["rot"].update(scaling=3))
    broken(lambda r: r["layers"][1]["mixer"].update(groups=2))              # of 3 heads
    broken(lambda r: r["layers"][1]["mixer"].update(norm_groups=5))         # of 48 values
    broken(lambda r: r["layers"][1]["mixer"].update(state=0))
    broken(lambda r: r["layers"][1]["mixer"].pop("conv"))
    broken(lambda r: r["layers"][2]["mixer"]["mask"].update(size=0))
    broken(lambda r: r["layers"][2]["mixer"].pop("kv_rank"))
    broken(lambda r: r["layers"][3]["mlp"].update(kind="moe"))
    broken(lambda r: r["layers"][3]["mlp"].pop("ff"))
    broken(lambda r: r["layers"][5].update(weights_of=8))                   # beyond the layers
    broken(lambda r: r["layers"][0].update(weights_of=5))                   # in a circle
    broken(lambda r: r["layers"][5].update(weights_of="l0"))


def test_parts_refuse_what_their_kernels_do_not_take():
    ctx = BuildContext(torch.float32, torch.device("meta"))
    for change in (dict(state=300), dict(conv=9)):
        raw = copy.deepcopy(tt.TG_A)
        raw["layers"][1]["mixer"].update(change)
        raw["layers"][6]["mixer"].update(change)
        with pytest.raises(ConfigError):
            DecoderModel(TigesunConfig.from_dict(raw).model_spec(), ctx)


@pytest.mark.parametrize("name", sorted(tt.CONFIGS))
def test_cache_and_state_needs(name):
    """Every run has one of its own, also those with another layer's tensors."""
    raw = tt.CONFIGS[name]
    model = DecoderModel(tt.config_of(name).model_spec(),
                         BuildContext(torch.float32, torch.device("meta")))
    needs = model.cache_needs()
    assert len(needs) == len(raw["layers"]) and None not in needs
    for L, need in zip(raw["layers"], needs):
        r = L["mixer"]
        if L["type"] == "attention":
            assert need == KVNeed(r["kv_heads"], r["dim"], None, value_dim=r["vdim"])
        elif L["type"] == "latent_attention":
            assert need == KVNeed(1, r["kv_rank"], (r["mask"] or {"size": None})["size"], value_dim=0)
        else:
            matrices = r["heads"] * r["vdim"] * ((r["state"] + 3) // 4 * 4)
            rows = (r["conv"] - 1) * (r["heads"] * r["vdim"] + 2 * r["groups"] * r["state"])
            assert need == StateNeed(((matrices + rows + 3) // 4 * 4,), torch.float32)


@pytest.mark.parametrize("name", sorted(tt.CONFIGS))
def test_declared_tensors(name):
    raw = tt.CONFIGS[name]
    W, V = raw["width"], raw["vocab"]
    d = declare_tensors(tt.config_of(name).model_spec())
    want = {"embed": (V, W), "embed.norm": (W,), "final.norm": (W,)}
    for i, L in enumerate(raw["layers"]):
        if L.get("weights_of") is not None:
            continue
        r, p = L["mixer"], f"l{i}."
        m = p + "mix."
        want.update({p + "norm1": (W,), p + "norm1b": (W,)})
        v = r["heads"] * r["vdim"]
        want[m + "o"] = (W, v)
        if L["type"] == "attention":
            G, d_ = r["kv_heads"], r["dim"]
            want.update({m + "q": (r["heads"] * d_, W), m + "k": (G * d_, W), m + "v": (G * r["vdim"], W),
                         m + "q.norm": (d_,), m + "k.norm": (d_,)})
        elif L["type"] == "latent_attention":
            k = r["kv_rank"]
            want.update({m + "q": (r["heads"] * r["dim"], W), m + "dkv": (k, W), m + "dkv.norm": (k,),
                         m + "uk": (r["heads"] * r["dim"], k), m + "uv": (v, k)})
        else:
            C, H = v + 2 * r["groups"] * r["state"], r["heads"]
            want.update({m + "in": (v + C + H, W), m + "conv": (C, r["conv"]), m + "conv.b": (C,),
                         m + "dt_bias": (H,), m + "A_log": (H,), m + "D": (H,), m + "norm": (v,)})
        if L["mlp"] is not None:
            ff = L["mlp"]["ff"]
            want.update({p + "norm2": (W,), p + "norm2b": (W,), p + "mlp.gate": (ff, W),
                         p + "mlp.gate.b": (ff,), p + "mlp.up": (ff, W), p + "mlp.up.b": (ff,),
                         p + "mlp.down": (W, ff), p + "mlp.down.b": (W,)})
    assert {n: t.shape for n, t in d.items() if not t.optional} == want
    assert {n for n, t in d.items() if t.optional} == {"head"}


def test_heads_a_workgroup_takes():
    """A divisor of a group's heads, more than one only while workgroups are left over."""
    for n_chunks in (1, 3, 16, 64):
        for H, G, dv in ((64, 1, 64), (128, 8, 64), (6, 2, 64), (12, 2, 128), (5, 5, 16), (4, 2, 200)):
            hb = ops.state_space_heads(n_chunks, H, G, dv)
            assert hb in (1, 2, 4) and (H // G) % hb == 0
            blocks = n_chunks * (H // hb) * ((dv + 63) // 64)
            assert hb == 1 or blocks >= ops.STATE_SPACE_WORKGROUPS
    assert ops.state_space_heads(64, 64, 1, 64) == 4 and ops.state_space_heads(1, 64, 1, 64) == 1


@pytest.mark.parametrize("name", ["A", "C"])
def test_a_folder_written_and_read(name, tmp_path):
    from zinfer_amd.config import load_config
    from zinfer_amd.weights.loader import load_tensors
    from zinfer_amd.weights.random_init import write_model_dir
    path = str(tmp_path / name)
    write_model_dir(path, tt.config_of(name), seed=3, dtype=torch.bfloat16)
    cfg = load_config(path)
    assert isinstance(cfg, TigesunConfig) and cfg.layers == tt.config_of(name).layers
    t = load_tensors(path, declare_tensors(cfg.model_spec()))
    assert t["l1.mix.in"].dtype == torch.bfloat16
    assert json.load(open(os.path.join(path, "config.json")))["architecture"] == "Tigesun"


# ------------------------------------------------------------------------------ the oracle by hand
def test_plain_masks():
    ok = P.seen(6, 2)
    assert [ok[i].nonzero().flatten().tolist() for i in (0, 1, 3, 5)] == [[0], [0, 1], [2, 3], [4, 5]]
    assert P.seen(5).tolist() == torch.ones(5, 5).tril().bool().tolist()
    q = torch.zeros(2, 1, 3, dtype=torch.float64)
    v = torch.tensor([[[2.0]], [[4.0]]], dtype=torch.float64)
    assert P.attend(q, q, v, 1.0, P.seen(2)).flatten().tolist() == [2.0, 3.0]


def test_plain_convolution():
    x = torch.tensor([[1.0], [2.0], [3.0]])
    y = P.causal_conv(x, torch.tensor([[10.0, 100.0]]), torch.tensor([0.5]))
    assert y.flatten().tolist() == [100.5, 210.5, 320.5]      # the last tap meets the token's own row


def test_plain_recurrence():
    """Two heads of one group: dt scales what is written, the decay is a half for dt = 1 with
    A = log log 2, D adds the token's own x."""
    T = 3
    x = torch.tensor([[[1.0], [1.0]], [[2.0], [1.0]], [[4.0], [1.0]]])
    B = torch.ones(T, 1, 1)
    C = torch.full((T, 1, 1), 2.0)
    dt = torch.tensor([[1.0, 1.0], [1.0, 0.0], [1.0, 2.0]])
    A = torch.full((2,), math.log(math.log(2.0)), dtype=torch.float64)
    y, S = P.state_space(x, B, C, dt, A, torch.tensor([0.0, 10.0]))
    assert torch.allclose(y[:, 0, 0], torch.tensor([2.0, 5.0, 10.5], dtype=torch.float64))
    # head 1: S = 1, 1 (dt 0 neither writes nor decays), then a quarter of it plus 2
    assert torch.allclose(y[:, 1, 0], torch.tensor([12.0, 12.0, 14.5], dtype=torch.float64))
    assert torch.allclose(S.flatten(), torch.tensor([5.25, 2.25], dtype=torch.float64))


def test_plain_gate_comes_before_the_norm_and_parts_are_normed_alone():
    y = torch.tensor([[3.0, 4.0, 1.0, 1.0]])
    z = torch.full((1, 4), 30.0)                               # silu(30) = 30
    n = P.gated_parts_norm(y, z, torch.tensor([1.0, 1.0, 1.0, 2.0]), 2, 0.0)
    r = math.sqrt(12.5)
    assert torch.allclose(n, torch.tensor([[3 / r, 4 / r, 1.0, 2.0]], dtype=torch.float64))
    a = P.gated_parts_norm(y, torch.tensor([[1.0, -1.0, 0.5, 2.0]]), torch.ones(4), 1, 0.0)
    assert float((a * a).mean()) == pytest.approx(1.0)


def test_plain_stretched_frequencies_and_rotation():
    # dims 4, base 10: pair numbers of t turns are 4 ln(100 / (2 pi t)) / (2 ln 10)
    f, length = P.stretched(10.0, 4, {"factor": 4.0, "original": 100, "fast": 16.0, "slow": 1.5})
    # fast: 2.00 * ln(0.995) / 2.30 = -0.004 -> 0;  slow: 2 * ln(10.6) / 2.30 = 2.05 -> 3
    want = [1.0, 10.0 ** -0.5 * (1.0 / 4.0 / 3.0 + 2.0 / 3.0)]
    assert f == pytest.approx(want) and length == pytest.approx(0.1 * math.log(4.0) + 1.0)
    z = torch.tensor([[[1.0, 7.0, 0.0, 5.0]]], dtype=torch.float64)
    r = P.rotate(z, torch.tensor([2]), {"dims": 2, "base": 10.0})      # the pair (0, 1) by 2 radians
    c, s = math.cos(2.0), math.sin(2.0)
    assert torch.allclose(r[0, 0], torch.tensor([c - 7 * s, 7 * c + s, 0.0, 5.0], dtype=torch.float64))


def test_plain_layers_share_tensors():
    raw, w = tt.TG_B, tt.weights_of("B")
    assert [P.owner(raw, i) for i in range(len(raw["layers"]))] == [6, 1, 2, 3, 4, 5, 6, 2, 2]
    toks = tt.tokens(12, raw["vocab"], 1)
    base, other = P.forward(toks, raw, w), dict(w)
    other["l6.mix.in"] = w["l6.mix.in"] * 1.5
    first, second = [], []
    P.forward(toks, raw, w, first)
    P.forward(toks, raw, other, second)
    assert float((first[0] - second[0]).abs().max()) > 1e-3     # the first layer runs with them, too
    assert base.shape == (12, raw["vocab"])
