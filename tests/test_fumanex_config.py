"""The Fumanex configuration on the CPU: what config.json gives, which layers mix their values,
what is refused, the cache or state each mixer asks for, the tensors a model declares, the
buckets of distances, a model folder written and read, and the plain implementation's own pieces
by hand."""
import copy
import json
import math
import os

import pytest
import torch

import fumanex_tiny as ft
import plain_fumanex as P
from zinfer_amd import ops
from zinfer_amd.config import (DenseMlpSpec, FixedDecayAttentionSpec, FumanexConfig,
                               MaskedGqaAttentionSpec, ParallelBlockSpec, RmsNormSpec, entry_for)
from zinfer_amd.config.distance import bucket_of_distances, bucket_starts
from zinfer_amd.errors import ConfigError
from zinfer_amd.models.build import declare_tensors
from zinfer_amd.models.decoder import DecoderModel
from zinfer_amd.parts.base import BuildContext, KVNeed, StateNeed


def test_registry_finds_the_family_by_its_one_name():
    assert entry_for(ft.FX_A).config_type is FumanexConfig
    assert entry_for({"architecture": "Fumanex", "model_type": "qwen3"}).config_type is FumanexConfig


@pytest.mark.parametrize("name", sorted(ft.CONFIGS))
def test_sizes_and_constants_come_from_the_file(name):
    raw = ft.CONFIGS[name]
    spec = ft.config_of(name).model_spec()
    eps = raw["norm"]["eps"]
    assert (spec.vocab_size, spec.hidden_size) == (raw["vocab"], raw["width"])
    assert spec.logit_scale == raw.get("logit_scale", 1.0) and not spec.tie_word_embeddings
    assert spec.embedding_multiplier == raw["embedding"]["scale"]
    assert spec.final_norm == RmsNormSpec(raw["width"], eps, weight_name="")
    assert [e.layer for e in spec.schedule] == list(range(len(raw["layers"])))
    mixing = 0
    for L, block in zip(raw["layers"], spec.layers):
        assert isinstance(block, ParallelBlockSpec) and block.ff_norm is None
        assert block.mixer_norm == RmsNormSpec(raw["width"], eps, weight_name="")
        m, r = block.mixer, L["mixer"]
        assert (m.n_heads, m.head_dim, m.value_dim) == (r["heads"], r["dim"], r["vdim"])
        if L["type"] == "attention":
            assert isinstance(m, MaskedGqaAttentionSpec)
            mask = r["mask"] or {"size": None, "keep_first": 0}
            assert (m.n_kv_heads, m.scale, m.softcap, m.window, m.keep_first, m.qk_unit_eps) == \
                (r["kv_heads"], r["scale"], r["softcap"], mask["size"], mask["keep_first"], eps)
            assert m.distance_bias.far == r["bias_max"] and m.bias and m.output_bias and m.sink
            assert m.rotary is None and m.chunk is None and m.qk_norm_eps is None
            assert m.value_mix == ("idle" if not r["v_mix"] else ("blend" if mixing else "source"))
            mixing += r["v_mix"]
        else:
            assert isinstance(m, FixedDecayAttentionSpec)
            assert list(m.decay) == r["decay"] and m.norm_eps == eps
            if L["type"] == "retention":
                assert (m.silu, m.norm, m.norm_name, m.gate) == (False, "head", None, "silu")
                assert m.k_scale == r["dim"] ** -0.5
                if r["rot"] is None:
                    assert m.rotary is None
                else:
                    assert m.rotary.dims == r["rot"]["dims"] and not m.rotary.interleaved
                    for i, f in enumerate(m.rotary.frequencies):
                        assert math.isclose(f, r["rot"]["base"] ** (-2.0 * i / r["rot"]["dims"]))
            else:
                assert (m.silu, m.norm, m.norm_name, m.gate) == (True, "row", "norm", "sigmoid")
                assert m.k_scale == 1.0 and m.rotary is None
        f = block.feed_forward
        if L["mlp"] is None:
            assert f is None
        else:
            assert isinstance(f, DenseMlpSpec) and f.activation == "gelu_tanh" and f.bias
            assert f.intermediate_size == L["mlp"]["ff"]


def test_what_the_configuration_refuses():
    def broken(change, base=ft.FX_A):
        raw = copy.deepcopy(base)
        change(raw)
        with pytest.raises(ConfigError):
            FumanexConfig.from_dict(raw)
    broken(lambda r: r.pop("vocab"))
    broken(lambda r: r.update(width=0))
    broken(lambda r: r["norm"].update(eps=-1.0))
    broken(lambda r: r.pop("norm"))
    broken(lambda r: r["embedding"].update(scale="big"))
    broken(lambda r: r.update(layers=[]))
    broken(lambda r: r["layers"][0].update(type="wkv"))
    broken(lambda r: r["layers"][0]["mixer"].update(kv_heads=4))            # of 6 heads
    broken(lambda r: r["layers"][0]["mixer"].pop("bias_max"))
    broken(lambda r: r["layers"][0]["mixer"].update(bias_max=0))
    broken(lambda r: r["layers"][0]["mixer"].update(softcap=0.0))
    broken(lambda r: r["layers"][0]["mixer"].update(v_mix=1))
    broken(lambda r: r["layers"][0]["mixer"]["mask"].update(size=0))
    broken(lambda r: r["layers"][0]["mixer"]["mask"].update(keep_first=-1))
    broken(lambda r: r["layers"][4]["mixer"].update(vdim=16))               # mixes with 3 x 20
    broken(lambda r: r["layers"][4]["mixer"].update(kv_heads=1))
    broken(lambda r: r["layers"][1]["mixer"].update(decay=[0.5, 0.5]))      # 3 heads
    broken(lambda r: r["layers"][1]["mixer"].update(decay=[0.5, 0.5, 1.5]))
    broken(lambda r: r["layers"][1]["mixer"].pop("decay"))
    broken(lambda r: r["layers"][1]["mixer"]["rot"].update(dims=5))
    broken(lambda r: r["layers"][1]["mixer"]["rot"].update(dims=22))
    broken(lambda r: r["layers"][1]["mixer"]["rot"].pop("base"))
    broken(lambda r: r["layers"][3]["mixer"].pop("vdim"))
    broken(lambda r: r["layers"][3]["mlp"].update(kind="moe"))
    broken(lambda r: r["layers"][3]["mlp"].pop("ff"))


@pytest.mark.parametrize("name", sorted(ft.CONFIGS))
def test_cache_and_state_needs(name):
    raw = ft.CONFIGS[name]
    spec = ft.config_of(name).model_spec()
    model = DecoderModel(spec, BuildContext(torch.float32, torch.device("meta")))
    for L, need in zip(raw["layers"], model.cache_needs()):
        r = L["mixer"]
        if L["type"] == "attention":
            mask = r["mask"] or {"size": None, "keep_first": 0}
            assert need == KVNeed(r["kv_heads"], r["dim"], mask["size"], value_dim=r["vdim"],
                                  keep_first=mask["keep_first"])
        else:
            padded = (r["dim"] + 3) // 4 * 4
            assert need == StateNeed((r["heads"] * r["vdim"] * padded,), torch.float32)


@pytest.mark.parametrize("name", sorted(ft.CONFIGS))
def test_declared_tensors(name):
    raw = ft.CONFIGS[name]
    W, V = raw["width"], raw["vocab"]
    d = declare_tensors(ft.config_of(name).model_spec())
    want = {"embed": (V, W), "head": (V, W), "final.norm": (W,)}
    for i, L in enumerate(raw["layers"]):
        r, p = L["mixer"], f"l{i}."
        want[p + "norm1"] = (W,)
        H, qk, v = r["heads"], r["heads"] * r["dim"], r["heads"] * r["vdim"]
        m = p + "mix."
        if L["type"] == "attention":
            G = r["kv_heads"]
            want.update({m + "q": (qk, W), m + "q.b": (qk,), m + "k": (G * r["dim"], W),
                         m + "k.b": (G * r["dim"],), m + "v": (G * r["vdim"], W),
                         m + "v.b": (G * r["vdim"],), m + "rel": (None, H), m + "vmix": (),
                         m + "sink": (H,), m + "o": (W, v), m + "o.b": (W,)})
        else:
            want.update({m + "q": (qk, W), m + "k": (qk, W), m + "v": (v, W), m + "g": (v, W),
                         m + "o": (W, v)})
            if L["type"] == "lightning":
                want[m + "norm"] = (v,)
        if L["mlp"] is not None:
            ff = L["mlp"]["ff"]
            want.update({p + "mlp.up": (ff, W), p + "mlp.up.b": (ff,), p + "mlp.down": (W, ff),
                         p + "mlp.down.b": (W,)})
    assert {n: t.shape for n, t in d.items()} == want
    # the share of the first values is needed by a layer that blends and by no other
    optional = {n for n, t in d.items() if t.optional}
    kinds = [getattr(b.mixer, "value_mix", None) for b in ft.config_of(name).model_spec().layers]
    assert optional == {f"l{i}.mix.vmix" for i, k in enumerate(kinds) if k in ("idle", "source")}


@pytest.mark.parametrize("buckets, far", [(32, 130), (32, 64), (8, 4.5), (8, 1000), (2, 3),
                                          (6, 128), (5, 9), (16, 8.25), (12, 6.001)])
def test_buckets_of_distances(buckets, far):
    """Against the plain rule for every distance up to far behind the last bucket's start, also
    where a distance lies exactly on a bucket's edge."""
    rows = bucket_of_distances(buckets, far)
    for n in range(3 * len(rows) + 40):
        assert rows[min(n, len(rows) - 1)] == P.bucket(n, buckets, far), n
    assert rows[-1] == buckets - 1 and (len(rows) == 1 or rows[-2] < buckets - 1)


def test_buckets_by_hand():
    # 8 rows, far 64: 0..3 alone; 4 * 16^(k/4) = 4, 8, 16, 32: powers of two sit on the edges
    assert bucket_starts(8, 64) == [0, 1, 2, 3, 4, 8, 16, 32]
    assert [P.bucket(n, 8, 64) for n in (3, 4, 7, 8, 15, 16, 31, 32, 1000)] == \
        [3, 4, 4, 5, 5, 6, 6, 7, 7]
    with pytest.raises(ConfigError):
        bucket_starts(8, 4)
    with pytest.raises(ConfigError):
        bucket_starts(1, 40)


def test_distance_table_layout():
    """The kernels' form: distances backwards between three more of the last and three zeros."""
    b = torch.tensor([[1.0, 2.0, 3.0], [4.0, 5.0, 6.0]])
    assert ops.distance_table(b).tolist() == [[3, 3, 3, 3, 2, 1, 0, 0, 0], [6, 6, 6, 6, 5, 4, 0, 0, 0]]


def test_chunk_lists():
    assert ops.fixed_decay_chunk_lists([1, 2, 32]) is None
    chunks, firsts, shorts = ops.fixed_decay_chunk_lists([1, 300, 5, 33, 128])
    assert chunks.tolist() == [[1, 1, 128, 0], [1, 129, 128, 0], [1, 257, 44, 0], [3, 306, 33, 0],
                               [4, 339, 128, 0]]
    assert firsts.tolist() == [[1, 0, 3], [3, 3, 1], [4, 4, 1]]
    assert shorts.tolist() == [0, 2]


def test_pages_of_a_request_with_kept_positions():
    from zinfer_amd.cache import CacheManager
    m = CacheManager([KVNeed(1, 4, 10, keep_first=9), KVNeed(1, 4, 10)], [None, None], 4, 40, 2,
                     torch.float32, "cpu")
    assert m.pages_at_most(1000, 8) == [(10 + 8 + 4 + 12 + 3) // 4, (10 + 8 + 4 + 3) // 4]
    m.add_request("a")
    for n in range(5, 101, 5):
        m.reserve("a", n)
        m.commit("a", n)
        held = [sum(p >= 0 for p in m.table(g, "a")) for g in range(2)]
        assert held[0] <= m.pages_at_most(100, 5)[0] and held[1] <= m.pages_at_most(100, 5)[1]
    assert all(p >= 0 for p in m.table(0, "a")[:3]) and m.table(0, "a")[3] < 0
    assert m.table(1, "a")[0] < 0
    m.release("a")
    m.check()


@pytest.mark.parametrize("name", ["A", "C"])
def test_a_folder_written_and_read(name, tmp_path):
    from zinfer_amd.config import load_config
    from zinfer_amd.weights.loader import load_tensors
    from zinfer_amd.weights.random_init import write_model_dir
    path = str(tmp_path / name)
    write_model_dir(path, ft.config_of(name), seed=3, dtype=torch.bfloat16)
    cfg = load_config(path)
    assert isinstance(cfg, FumanexConfig) and cfg.layers == ft.config_of(name).layers
    t = load_tensors(path, declare_tensors(cfg.model_spec()))
    assert t["l1.mix.q"].dtype == torch.bfloat16
    assert json.load(open(os.path.join(path, "config.json")))["architecture"] == "Fumanex"


# ------------------------------------------------------------------------------ the oracle by hand
def test_plain_masks_and_sink():
    ok = P.seen(7, 2, 1)
    assert [ok[i].nonzero().flatten().tolist() for i in (0, 1, 3, 6)] == [[0], [0, 1], [0, 2, 3], [0, 5, 6]]
    assert P.seen(5, None, 0).tolist() == torch.ones(5, 5).tril().bool().tolist()
    a = P.sink_softmax(torch.zeros(1, 2, 2, dtype=torch.float64), P.seen(2, None, 0),
                       torch.tensor([math.log(2.0)]))
    assert torch.allclose(a[0], torch.tensor([[1 / 3, 0], [0.25, 0.25]], dtype=torch.float64))


def test_plain_recurrence_and_rotation():
    q = torch.ones(3, 1, 1)
    k = torch.tensor([1.0, 2.0, 3.0]).view(3, 1, 1)
    v = torch.ones(3, 1, 1)
    o, S = P.decayed_sums(q, k, v, [0.5])
    assert o.flatten().tolist() == [1.0, 2.5, 4.25] and S.item() == 4.25
    z = torch.tensor([[[1.0, 7.0, 0.0, 5.0]]], dtype=torch.float64)
    r = P.rotate(z, torch.tensor([2]), 2, 10.0)             # the pair (0, 1) by 2 radians
    c, s = math.cos(2.0), math.sin(2.0)
    assert torch.allclose(r[0, 0], torch.tensor([c - 7 * s, 7 * c + s, 0.0, 5.0], dtype=torch.float64))


def test_plain_first_layer_that_mixes_leaves_its_values():
    """The first mixing layer's output does not read its own share; a later one's does."""
    raw, w = ft.FX_A, ft.weights_of("A")
    toks = ft.tokens(12, raw["vocab"], 1)
    base = P.forward(toks, raw, w)
    for layer, moves in ((0, False), (2, False), (4, True)):
        other = dict(w)
        other[f"l{layer}.mix.vmix"] = w[f"l{layer}.mix.vmix"] + 0.5
        assert bool((P.forward(toks, raw, other) - base).abs().max() > 1e-3) is moves
