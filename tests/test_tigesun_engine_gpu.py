"""Tigesun models through the engine against ``plain_tigesun``, in 32-bit and in bfloat16: whole
prompts; most of a prompt and then its last tokens one by one; portions of changing size down to
two tokens; token by token from the first token on (long decoding); mixed batches of four live
requests in a pool so small that pages are used again (what was given back is overwritten with
NaN first) with four state slots that are used again; the same bits however a prompt is cut in
32-bit; a slot used again starts from zero; a request longer than the pool of its windows; every
run of a layer alone; a token at both sides of the window's edge, and one far back that only the
attention or only the state space can still see; a feed-forward whose bias a norm takes in; greedy
generation through the entry point and the scheduler; decode steps replayed as graphs; the replay
program and the command line on a model folder."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

import plain_tigesun as P
import tigesun_tiny as tt
import traces
from gpu_util import DEV

pytestmark = pytest.mark.gpu

# float32: what is left is the order of sums and the 32-bit angles, decays and exponentials.
# bfloat16: activations are rounded to 8 bits of mantissa some ten times a layer; a norm behind
# every sublayer gives a small output full weight, its rounding with it.
TOL = {"float32": 5e-5, "bfloat16": 0.075}
LENGTHS = {"A": (1, 5, 23, 60, 150), "B": (2, 9, 47, 130), "C": (3, 17, 64), "D": (4, 33, 100, 260)}
_ref = {}


def _requests(name, twice=False):
    vocab = tt.CONFIGS[name]["vocab"]
    req = {f"r{i}": tt.tokens(n, vocab, 100 + i) for i, n in enumerate(LENGTHS[name])}
    if twice:
        req.update({f"s{i}": tt.tokens(n, vocab, 200 + i)
                    for i, n in enumerate(reversed(LENGTHS[name]))})
    return req


def _reference(name, requests):
    w = None
    out = {}
    for rid, toks in requests.items():
        key = (name, tuple(toks))
        if key not in _ref:
            w = w or tt.weights_of(name)
            _ref[key] = P.forward(toks, tt.CONFIGS[name], w).numpy()
        out[rid] = _ref[key]
    return out


def _engine(name, dtype, num_pages, poison=True, max_requests=4, use_graphs=True, weights=None):
    from zinfer_amd.engine import Engine
    from zinfer_amd.models.build import build_model
    store = torch.float32 if dtype == "float32" else torch.bfloat16
    w = weights if weights is not None else tt.weights_of(name, dtype=store)
    model = build_model(tt.config_of(name).model_spec(), w, dtype, DEV)
    return Engine(model, page_size=tt.PAGE_SIZE[name], num_pages=num_pages,
                  max_requests=max_requests, poison_freed=poison, use_graphs=use_graphs)


def _replay(eng, steps):
    from zinfer_amd.engine import StepEntry
    outputs = {}
    for st in steps:
        for e in st["entries"]:
            held = eng.length(e["id"]) if eng.has_request(e["id"]) else 0
            assert e["start"] == held
        logits = eng.step([StepEntry(e["id"], e["tokens"], e["want"]) for e in st["entries"]],
                          end=st["end"])
        if logits.shape[0]:
            outputs[st["step"]] = logits.cpu().numpy().copy()
    eng.cache.check()
    assert not eng.cache.requests
    return outputs


def _compare(steps, outputs, ref, vocab, dtype):
    """Every position within the tolerance in 32-bit.  In bfloat16 a token whose output of a state
    space nearly vanishes in one of the normed parts brings its rounding in with full weight: one
    position in thirty may lie beyond the tolerance, none beyond three times it, and the median
    lies within half of it."""
    tolerance = TOL[dtype]
    got = traces.collect(steps, outputs, vocab)
    assert set(got) == set(ref)
    errs = []
    for rid in ref:
        assert got[rid].shape == ref[rid].shape
        assert np.isfinite(got[rid]).all(), f"{rid}: logits are not finite"
        err = np.abs(got[rid].astype(np.float64) - ref[rid]).max(axis=1) / np.abs(ref[rid]).max()
        bad = np.nonzero(err > (tolerance if dtype == "float32" else 3 * tolerance))[0]
        assert bad.size == 0, \
            (f"request {rid}: {bad.size} of {len(err)} positions wrong, the first {bad[0]} "
             f"(error {err[bad[0]]:.3g} > {tolerance})")
        errs.append(err)
    errs = np.concatenate(errs)
    if dtype == "bfloat16":
        assert float(np.median(errs)) <= tolerance / 2, float(np.median(errs))
        assert (errs > tolerance).sum() <= len(errs) / 30 + 1, (errs > tolerance).sum()
    return float(errs.max())


MODES = {"whole": traces.whole,
         "prefill_then_single": lambda r: traces.prefill_then_single(r, tail=20),
         "portions": traces.changing_portions, "token_by_token": traces.token_by_token,
         "mixed": lambda r: traces.mixed(r, decode_tail=9)}


@pytest.mark.parametrize("mode", list(MODES))
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", sorted(tt.CONFIGS))
def test_replay_modes(name, dtype, mode):
    requests = _requests(name, twice=mode == "mixed")
    steps = MODES[mode](requests)
    page = tt.PAGE_SIZE[name]
    # the pool holds what is live at the fullest step and no more; four state slots
    pages = (traces.peak_tokens(steps, page) + page - 1) // page
    eng = _engine(name, dtype, pages)
    outputs = _replay(eng, steps)
    worst = _compare(steps, outputs, _reference(name, requests), tt.CONFIGS[name]["vocab"], dtype)
    if mode == "mixed":
        assert max(len(st["entries"]) for st in steps) == 4
        assert len(requests) > 4                     # so every slot served several requests
        for grp in eng.cache.groups:
            assert grp.pages.handed_out > grp.pages.num_pages, "no page was used again"
    print(f"{name} {dtype} {mode}: error {worst:.3g}")


@pytest.mark.parametrize("name", sorted(tt.CONFIGS))
def test_cut_and_batch_leave_the_bits(name):
    """32-bit: a position's logits are the same bits whole, in portions, token by token and
    beside other requests, whichever slot and pages the request got."""
    requests = _requests(name)
    vocab = tt.CONFIGS[name]["vocab"]
    rows = []
    for mode in ("whole", "portions", "token_by_token", "mixed"):
        steps = MODES[mode](requests)
        eng = _engine(name, "float32", 64, poison=False)
        rows.append(traces.collect(steps, _replay(eng, steps), vocab))
    for other in rows[1:]:
        for rid in rows[0]:
            assert np.array_equal(rows[0][rid], other[rid]), rid


def test_a_slot_that_is_used_again_starts_from_zero():
    """Two requests one after the other in an engine with a single state slot: the second one's
    logits are those it has alone in a fresh engine (32-bit, the same bits): neither the
    matrices nor the convolutions' last rows of the first request are left."""
    name = "A"
    vocab = tt.CONFIGS[name]["vocab"]
    a, b = tt.tokens(40, vocab, 11), tt.tokens(33, vocab, 12)
    eng = _engine(name, "float32", 8, max_requests=1)
    first = _replay(eng, traces.changing_portions({"a": a}, sizes=(9, 2, 11)))
    again = _replay(eng, traces.changing_portions({"b": b}, sizes=(5, 28)))
    fresh = _replay(_engine(name, "float32", 8, max_requests=1),
                    traces.changing_portions({"b": b}, sizes=(5, 28)))
    assert first and set(again) == set(fresh)
    for k in fresh:
        assert np.array_equal(again[k], fresh[k])


def test_a_request_longer_than_the_pool_of_its_windows():
    """A model of windowed latent layers and a state space: a request of 150 tokens in a pool of
    64, whose windows' pages are given back on the way (and overwritten with NaN)."""
    from zinfer_amd.config import TigesunConfig
    from zinfer_amd.engine import Engine
    from zinfer_amd.models.build import build_model
    raw = dict(tt.TG_C, layers=[tt.TG_C["layers"][i] for i in (0, 1)] + [dict(tt.TG_C["layers"][0])])
    raw["layers"][2] = dict(raw["layers"][0], weights_of=0)
    toks = tt.tokens(150, raw["vocab"], 31)
    w = tt.weights_for(raw)
    model = build_model(TigesunConfig.from_dict(raw).model_spec(), w, "float32", DEV)
    eng = Engine(model, page_size=4, num_pages=16, max_requests=1, poison_freed=True)
    steps = traces.changing_portions({"r": toks}, sizes=(7, 2, 13, 1, 5))
    got = traces.collect(steps, _replay(eng, steps), raw["vocab"])["r"]
    want = P.forward(toks, raw, w).numpy()
    assert float(np.abs(got - want).max() / np.abs(want).max()) < TOL["float32"]
    assert all(g.pages.high_water <= 16 < g.pages.handed_out for g in eng.cache.groups)


def test_every_run_of_a_layer_alone():
    """Every layer's own tensors alone (``Engine.probe_block``) on the plain implementation's
    stream before a run gives the plain implementation's stream after it, in 32-bit; and the
    whole model's stream behind every run (the decoder's probe) is the plain one."""
    from zinfer_amd.engine import StepEntry
    for name in ("A", "B", "C"):
        raw = tt.CONFIGS[name]
        toks = tt.tokens(50, raw["vocab"], 3)
        w = tt.weights_of(name)
        streams = []
        P.forward(toks, raw, w, streams)
        eng = _engine(name, "float32", 64, poison=False)
        before = P.embedding(toks, raw, w)
        for index, after in zip(tt.config_of(name).order, streams):
            got, held = eng.probe_block(index, before.to(torch.float32).to(DEV))
            assert held == len(toks)
            err = float((got.cpu().double() - after).abs().max() / after.abs().max())
            assert err < 2e-5, f"{name} layer {index}: {err:.3g}"
            before = after
        seen = []
        eng.model.layer_probe = lambda pos, x: seen.append(x.detach().cpu().double())
        eng.step([StepEntry("r", toks, [])], end=["r"])
        eng.model.layer_probe = None
        assert len(seen) == len(streams)
        for pos, (got, want) in enumerate(zip(seen, streams)):
            err = float((got - want).abs().max() / want.abs().max())
            assert err < 5e-5, f"{name} run {pos}: {err:.3g}"


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("decoded", [1, 40])
def test_a_token_shows_inside_the_window_and_not_outside(dtype, decoded):
    """One latent layer with a window of 9 whose queries and latents are the token's own
    direction: a token that repeats the last one takes nearly all the weight.  As the window's
    oldest it shows in the logits, one further back it does not; in a prompt and behind 40 single
    tokens."""
    from zinfer_amd.config import TigesunConfig
    from zinfer_amd.engine import Engine, StepEntry
    from zinfer_amd.models.build import build_model
    W, V, n = 16, 40, 120
    L = {"type": "latent_attention", "mlp": None,
         "mixer": {"heads": 1, "dim": 16, "vdim": 16, "kv_rank": 16, "scale": 1.0, "mask": {"size": 9}}}
    raw = {"architecture": "Tigesun", "vocab": V, "width": W, "norm": {"eps": 1e-6}, "layers": [L]}
    eye, ones = torch.eye(W), torch.ones(W)
    w = {"embed": torch.zeros(V, W), "embed.norm": ones, "final.norm": ones, "l0.norm1": ones,
         "l0.norm1b": ones, "l0.mix.q": eye, "l0.mix.dkv": eye, "l0.mix.dkv.norm": ones,
         "l0.mix.uk": eye, "l0.mix.uv": torch.zeros(W, W), "l0.mix.o": eye.clone()}
    w["embed"][0, 0] = 1.0                         # the filler's direction
    w["embed"][1, 1] = 1.0                         # the query's
    w["embed"][2, 1], w["embed"][2, 2] = 1.0, 0.5  # the planted token: the query's, and a mark
    w["embed"][3, 5] = 1.0                         # whose value the logit of token 3 reads
    w["l0.mix.uv"][5, 2] = 1.0
    w["l0.mix.uv"][6, 0] = w["l0.mix.uv"][7, 1] = 1.0     # what the others bring
    store = torch.float32 if dtype == "float32" else torch.bfloat16
    w = {k: v.to(store) for k, v in w.items()}
    model = build_model(TigesunConfig.from_dict(raw).model_spec(), w, dtype, DEV)
    for at, seen in ((n - 9, True), (n - 10, False), (n - 2, True), (0, False), (60, False)):
        eng = Engine(model, page_size=4, num_pages=40, max_requests=1, poison_freed=True)
        toks = [0] * n
        toks[at], toks[-1] = 2, 1
        head = n - decoded
        eng.step([StepEntry("r", toks[:head], [])])
        for p in range(head, n):
            logits = eng.step([StepEntry("r", [toks[p]], [0])])
        mark = float(logits[0, 3])
        want = float(P.forward(toks, raw, w)[-1, 3])
        assert abs(mark - want) < (1e-4 if dtype == "float32" else 0.03)
        assert (mark > 0.1) is seen, (at, mark)


def _silenced(raw, quiet):
    """Weights in which the mixers of the kinds ``quiet`` bring nothing (the gain of the norm
    behind them is zero)."""
    w = tt.weights_for(raw)
    for i, L in enumerate(raw["layers"]):
        if L["type"] in quiet and L.get("weights_of") is None:
            w[f"l{i}.norm1b"] = torch.zeros_like(w[f"l{i}.norm1b"])
    return w


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("kind", ["attention", "mamba2"])
def test_a_token_far_back_shows_through_either_mixer(kind, dtype):
    """Two prompts of 300 tokens that differ in token 2 alone, with every other kind of mixer
    silent: only the attention (its keys lie 19 pages back) or only the state spaces' slow heads
    still know it.  The last position's logits differ between the prompts, and the engine's
    difference is the plain implementation's: in one step, and with the last 40 tokens decoded
    one by one."""
    raw = tt.TG_A
    w = _silenced(raw, {"attention", "latent_attention", "mamba2"} - {kind})
    if kind == "mamba2":
        for i in (1, 3):
            w[f"l{i}.mix.A_log"] = torch.full_like(w[f"l{i}.mix.A_log"], -9.0)
    a = tt.tokens(300, raw["vocab"], 77)
    b = list(a)
    b[2] = (a[2] + 1) % raw["vocab"]
    ref = {k: P.forward(t, raw, w)[-1].numpy() for k, t in (("a", a), ("b", b))}
    gap = np.abs(ref["a"] - ref["b"]).max()
    assert gap > 1e-3 * np.abs(ref["a"]).max()          # the far token matters
    store = torch.float32 if dtype == "float32" else torch.bfloat16
    wd = {n: t.to(store) for n, t in w.items()}
    for mode in (traces.whole, lambda r: traces.prefill_then_single(r, tail=40)):
        got = {}
        for k, t in (("a", a), ("b", b)):
            steps = mode({k: t})
            eng = _engine("A", dtype, 32, weights=wd)
            got[k] = traces.collect(steps, _replay(eng, steps), raw["vocab"])[k][-1]
        if dtype == "float32":
            assert np.abs((got["a"] - got["b"]) - (ref["a"] - ref["b"])).max() < 0.02 * gap
        else:
            assert np.abs(got["a"] - got["b"]).max() > 0.3 * gap


def test_a_norm_that_takes_the_bias_in_gives_what_a_bias_added_before_gives():
    """The feed-forward's output bias inside the closing norm's kernel against the bias added to
    the sublayer's rows by a kernel of its own, 32-bit: the same to rounding."""
    from zinfer_amd.parts.mlp import GatedMlp
    requests = _requests("A")
    steps, vocab = traces.changing_portions(requests), tt.CONFIGS["A"]["vocab"]
    inside = traces.collect(steps, _replay(_engine("A", "float32", 80), steps), vocab)
    try:
        GatedMlp.leaves_bias = False
        apart = traces.collect(steps, _replay(_engine("A", "float32", 80), steps), vocab)
    finally:
        GatedMlp.leaves_bias = True
    for rid in inside:
        scale = float(np.abs(apart[rid]).max())
        assert float(np.abs(inside[rid] - apart[rid]).max()) < 2e-5 * scale, rid


def _write_folder(name, path, store):
    from zinfer_amd.weights.safetensors_io import write_safetensors
    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(tt.CONFIGS[name], f)
    write_safetensors(os.path.join(path, "model.safetensors"), tt.weights_of(name, dtype=store))
    return path


def _check_greedy(name, prompt, got, w):
    logits = P.forward(list(prompt) + list(got), tt.CONFIGS[name], w)
    for i, tok in enumerate(got):
        row = logits[len(prompt) - 1 + i]
        top2 = torch.topk(row, 2).values
        if float(top2[0] - top2[1]) > 1e-3 * float(row.abs().max()):
            assert int(row.argmax()) == tok, f"token {i} of a prompt of {len(prompt)}"


@pytest.mark.parametrize("name", ["B", "D"])
def test_greedy_generation_through_entry_point_and_scheduler(name, tmp_path):
    """Prompts of unequal length generate together (more prompts than state slots, so slots
    are used again); every request's tokens are the plain implementation's arg-max wherever
    that one is clear."""
    from zinfer_amd.entrypoints import LLM, SamplingParams
    path = _write_folder(name, str(tmp_path / name), torch.float32)
    vocab = tt.CONFIGS[name]["vocab"]
    prompts = [tt.tokens(n, vocab, 300 + n) for n in (3, 41, 18, 7, 29, 12)]
    llm = LLM(path, dtype="float32", device=DEV, page_size=tt.PAGE_SIZE[name], max_tokens=512,
              max_step_tokens=48, chunk_size=16, max_seqs=4)
    n_new = 14
    outs = llm.generate(prompts, SamplingParams(temperature=0.0, max_new_tokens=n_new,
                                                ignore_eos=True))
    w = tt.weights_of(name)
    for prompt, got in zip(prompts, outs):
        assert len(got) == n_new
        _check_greedy(name, prompt, got, w)


def test_decode_steps_replayed_as_graphs_keep_the_state_right():
    """32-bit: prompt, then forty single tokens through captured graphs (the first step of a
    shape runs once eagerly before it is captured and replayed: matrices and last rows must
    not move twice), against the same without graphs: the same bits."""
    name = "A"
    toks = tt.tokens(70, tt.CONFIGS[name]["vocab"], 21)
    steps = traces.prefill_then_single({"r": toks}, tail=40)
    with_graphs = _engine(name, "float32", 16, poison=False, use_graphs=True)
    a = _replay(with_graphs, steps)
    b = _replay(_engine(name, "float32", 16, poison=False, use_graphs=False), steps)
    assert with_graphs.graph_replays > 30
    for k in b:
        assert np.array_equal(a[k], b[k]), k


def test_long_generation_in_bfloat16_stays_finite_and_uses_graphs(tmp_path):
    """Sixty tokens decoded behind a prompt through the scheduler's runs of decode steps: the
    steps replay as graphs and the tokens are ids."""
    from zinfer_amd.entrypoints import LLM, SamplingParams
    name = "D"
    path = _write_folder(name, str(tmp_path / name), torch.bfloat16)
    prompts = [tt.tokens(n, 512, 400 + n) for n in (5, 70)]
    params = SamplingParams(temperature=0.0, max_new_tokens=60, ignore_eos=True)
    llm = LLM(path, dtype="bfloat16", device=DEV, page_size=16, max_tokens=512, max_seqs=4)
    outs = llm.generate(prompts, params)
    assert all(len(o) == 60 and all(0 <= t < 512 for t in o) for o in outs)
    assert llm.engine.graph_replays > 0


def test_replay_program_on_a_model_folder(tmp_path):
    """``bin/trace_run`` chooses the model class by config.json and writes the logits of a
    mixed trace; both dtypes."""
    name = "C"
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    requests = _requests(name, twice=True)
    steps = traces.mixed(requests, decode_tail=5)
    text = "".join(json.dumps({k: v for k, v in st.items()}) + "\n" for st in steps)
    ref = _reference(name, requests)
    for dtype in ("float32", "bfloat16"):
        store = torch.float32 if dtype == "float32" else torch.bfloat16
        path = _write_folder(name, str(tmp_path / dtype), store)
        out = str(tmp_path / ("out_" + dtype))
        r = subprocess.run([sys.executable, os.path.join(root, "bin", "trace_run"), "--model", path,
                            "--dtype", dtype, "--out", out, "--max-tokens",
                            str(traces.peak_tokens(steps, 64))],
                           input=text, capture_output=True, text=True, timeout=300)
        assert r.returncode == 0, r.stderr[-2000:]
        done = [l for l in r.stdout.splitlines() if l.startswith("done ")]
        assert done == [f"done {st['step']}" for st in steps]
        outputs = {st["step"]: np.fromfile(os.path.join(out, f"{st['step']}.f32"), dtype="<f4")
                   for st in steps if any(e["want"] for e in st["entries"])}
        _compare(steps, outputs, ref, tt.CONFIGS[name]["vocab"], dtype)


def test_generation_through_the_command_line(tmp_path):
    """``bin/zinfer generate-token-ids`` on a Tigesun folder: the oracle's greedy tokens."""
    name = "A"
    path = _write_folder(name, str(tmp_path / name), torch.float32)
    prompt = tt.tokens(11, tt.CONFIGS[name]["vocab"], 9)
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    r = subprocess.run([sys.executable, os.path.join(root, "bin", "zinfer"), "generate-token-ids",
                        path, ",".join(map(str, prompt)), "6", "--dtype", "float32"],
                       capture_output=True, text=True, timeout=300)
    assert r.returncode == 0, r.stderr[-2000:]
    line = [l for l in r.stdout.splitlines() if l.startswith("tokens: ")][0]
    got = json.loads(line[len("tokens: "):])
    assert got[:len(prompt)] == prompt and len(got) == len(prompt) + 6
    _check_greedy(name, prompt, got[len(prompt):], tt.weights_of(name))
