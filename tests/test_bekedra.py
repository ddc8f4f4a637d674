"""Bekedra through the engine and op by op, against the plain oracle in tests/bekedra_oracle.py.

Every test builds its own small configuration and random weights (sizes all different from one another and from any
shipped checkpoint), writes them as a checkpoint, loads that through the engine, and compares with the oracle.  The CPU
runs use the torch reference ops, the ``gpu`` ones the HIP kernels; float32 comparisons are tight (rounding only),
bfloat16 ones use the spread that bf16 rounding gives.  A dictated step goes through LLMEngine.replay_step, i.e. the
scheduler, the block manager, the runner's packed metadata (and decode hipGraphs on the GPU) and model.forward.
"""
from __future__ import annotations

import copy
import dataclasses
import os
import sys

import pytest
import torch

sys.path.insert(0, os.path.dirname(os.path.abspath(__file__)))
import bekedra_oracle as O  # noqa: E402

from symmetry_amd import ops  # noqa: E402
from symmetry_amd.engine.llm_engine import EngineConfig, LLMEngine  # noqa: E402
from symmetry_amd.engine.sequence import SamplingParams  # noqa: E402
from symmetry_amd.models import config as C  # noqa: E402
from symmetry_amd.models.weights import bekedra_random_weights, save_bekedra_checkpoint  # noqa: E402

DEVICES = ["cpu", pytest.param("cuda", marks=pytest.mark.gpu)]
F64, BF16, F32 = torch.float64, torch.bfloat16, torch.float32
CAUSAL = 1 << 30


def say(*a):
    print(*a, flush=True)


# ---- configurations ---------------------------------------------------------------------------------------------
def keyv(heads=6, kv=2, dim=10, scale=0.4, coef=0.3, every=7):
    return C.NormedAttnSpec(heads, kv, dim, dim, scale, row_norm=True, bias=True, key_values=True, temp_coef=coef,
                            temp_every=every)


def rotary(heads=4, kv=4, dim=14, vdim=9, scale=0.5, dims=6, base=200.0, scaling=(3.0, 1.0, 5.0, 60.0), cap=4.0):
    rot = C.RotarySpec(dims, base, half=True,
                       **(dict(zip(("factor", "low", "high", "original"), scaling)) if scaling else {}))
    return C.NormedAttnSpec(heads, kv, dim, vdim, scale, rot=rot, softcap=cap, sink=True, gate=True)


def lay(kind, mixer, ff=None):
    return C.BekedraLayer(kind, mixer, C.ChosenSoftmaxSpec(*ff) if ff else None)


def cfg_mixed(width=40, vocab=67):
    """Every branch once: both mixers inside and outside the loop (so every pass has planes of its own), shared and own key
    heads, value heads of another size than the keys, layers without feed-forward (one of them the loop's last), 1 / 2 / 3
    experts per token and all of them, frequency scaling with and without, part of a head and all of it turning."""
    layers = (
        lay("attention_2", rotary(), (7, 3, 20)),
        lay("attention", keyv(), (5, 2, 28)),
        lay("attention_2", rotary(heads=6, kv=3, dim=8, vdim=21, dims=8, scaling=None, cap=9.0), (4, 1, 12)),
        lay("attention", keyv(heads=3, kv=3, dim=17, coef=1.5, every=1)),
        lay("attention", keyv(heads=4, kv=1, dim=6, coef=0.2, every=33), (3, 3, 36)),
        lay("attention_2", rotary(heads=2, kv=1, dim=24, vdim=5, dims=2, base=30.0), None),
    )
    return C.BekedraConfig(name="t-mixed", vocab_size=vocab, hidden_size=width, layers=layers, loop=C.LoopSpec(1, 4, 3),
                           embed_scale=3.0, norm_eps=1e-5)


def cfg_tiled(width=64, vocab=97):
    """Sizes that the prompt kernel, the vectorised row kernels, the MFMA router and both expert kernels take; the loop over
    all layers but the last."""
    layers = (
        lay("attention_2", rotary(heads=4, kv=2, dim=32, vdim=32, dims=16, scale=0.3, base=1000.0,
                                  scaling=(8.0, 1.0, 4.0, 200.0), cap=6.0), (10, 3, 64)),
        lay("attention", keyv(heads=6, kv=3, dim=48, scale=0.2, coef=0.4, every=20), (20, 4, 96)),
        lay("attention", keyv(heads=4, kv=4, dim=64, scale=0.15, coef=0.1, every=50)),
        lay("attention_2", rotary(heads=3, kv=1, dim=80, vdim=80, dims=80, scale=0.2, base=500.0, scaling=None, cap=3.0),
            (40, 2, 32)),
    )
    return C.BekedraConfig(name="t-tiled", vocab_size=vocab, hidden_size=width, layers=layers, loop=C.LoopSpec(0, 3, 2),
                           embed_scale=6.0, norm_eps=1e-6)


def cfg_plain(width=24, vocab=50):
    """The values at which mechanisms vanish or coincide: one pass, one head, one expert, embedding scale one, no frequency
    scaling, a temperature that never moves, a cap far above every score."""
    layers = (lay("attention", keyv(heads=1, kv=1, dim=8, scale=1.0, coef=0.0, every=1000), (1, 1, 8)),
              lay("attention_2", rotary(heads=1, kv=1, dim=8, vdim=8, dims=8, scale=1.0, scaling=None, cap=1000.0)),
              lay("attention_2", rotary(heads=2, kv=2, dim=4, vdim=4, dims=2, scale=1.0, scaling=None), (2, 2, 24)))
    return C.BekedraConfig(name="t-plain", vocab_size=vocab, hidden_size=width, layers=layers, loop=C.LoopSpec(1, 2, 1),
                           embed_scale=1.0, norm_eps=1e-5)


def cfg_noloop():
    return dataclasses.replace(cfg_plain(width=28), name="t-noloop", loop=None)


def cfg_loop_to_the_end():
    """The loop covers the last layer, so the output norm follows a pass."""
    return dataclasses.replace(cfg_plain(width=20), name="t-loopend", loop=C.LoopSpec(1, 3, 4), embed_scale=0.7)


ALL = [cfg_mixed, cfg_tiled, cfg_plain, cfg_noloop, cfg_loop_to_the_end]


def checkpoint(cfg, tmp_path, seed=0, sharpen=None):
    """(routers are scaled to be decisive: a choice that bf16 rounding flips would be another function)"""
    w = bekedra_random_weights(cfg, seed=seed)
    for k in w.tensors:
        if k.endswith("mlp.router"):
            w.tensors[k] = w.tensors[k] * 4.0
    if sharpen:
        sharpen(w.tensors)
    path = str(tmp_path / f"{cfg.name}-{seed}")
    save_bekedra_checkpoint(w, path)
    return path, C.bekedra_to_config(cfg), {k: v.to(BF16) for k, v in w.tensors.items()}


def engine(path, device, dtype, blocks=24, seqs=4, block_size=16, graphs=True, pipeline=False, prefix=False):
    return LLMEngine(EngineConfig(model="t", weights=path, dtype=dtype, device=device, max_num_seqs=seqs,
                                  block_size=block_size, num_kv_blocks=blocks + 1, max_model_len=blocks * block_size,
                                  max_num_batched_tokens=8192, use_graphs=graphs, enable_prefix_caching=prefix,
                                  pipeline=pipeline))


def tokens(n, vocab, seed):
    g = torch.Generator().manual_seed(seed)
    return torch.randint(0, vocab, (n,), generator=g).tolist()


def run_schedule(eng, prompts: dict, schedule: list) -> dict:
    """schedule: steps of [(request, tokens this step)]; every position's logits are asked for.  -> id -> [n, V]."""
    at = {r: 0 for r in prompts}
    got = {r: [] for r in prompts}
    for step in schedule:
        entries, ends = [], []
        for r, n in step:
            lo = at[r]
            entries.append((r, prompts[r][lo:lo + n], list(range(n))))
            at[r] = lo + n
            if at[r] == len(prompts[r]):
                ends.append(r)
        lg = eng.replay_step(entries, ends)
        o = 0
        for r, n in step:
            got[r].append(lg[o:o + n].clone())
            o += n
    return {r: torch.cat(v) for r, v in got.items() if v}


def err(a, b, dtype="float32"):
    """The worst row's distance in units of the logits' spread; in bfloat16 the distance that nine rows in ten keep (a token
    whose router hesitates between two experts may take the other one)."""
    d = a.double() - b.double()
    d = d - d.mean(-1, keepdim=True)
    e = d.pow(2).mean(-1).sqrt() / b.double().std(-1).clamp_min(1e-6)
    return float(e.max() if dtype == "float32" else e.quantile(0.9))


TOL = {"float32": 2e-4, "bfloat16": 0.1}    # bf16: a lost mechanism gives errors near 1 in most rows


def oracle_logits(cj, W, toks):
    return O.forward(cj, W, toks).float()


def _sharp(t):
    """Attention that looks hard at single keys, sinks that matter: a lost key or a dropped sink moves the logits by far more
    than the tolerance."""
    for k in t:
        if k.endswith("mix.q.norm"):
            t[k] = t[k] * 3.0
        if k.endswith("sink"):
            t[k] = t[k] + 2.0


# ---- the whole model through the engine ------------------------------------------------------------------------------
@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("make", ALL)
def test_prompt_decode_portions(tmp_path, device, dtype, make):
    """Whole prompt, prompt then token-by-token decoding, portions down to two tokens, and token by token from the first
    token all give the oracle's logits."""
    say("prompt/decode/portions", make.__name__, device, dtype)
    cfg = make()
    path, cj, W = checkpoint(cfg, tmp_path, seed=1)
    toks = tokens(75, cfg.vocab_size, 1)
    want = oracle_logits(cj, W, toks)
    eng = engine(path, device, dtype)
    for name, cuts in (("whole", [75]), ("decode", [30] + [1] * 45), ("portions", [2, 3, 17, 2, 16, 1, 1, 5, 2, 26]),
                       ("tokens", [1] * 24)):
        say("  ", name)
        n = sum(cuts)
        got = run_schedule(eng, {"a": toks[:n]}, [[("a", c)] for c in cuts])["a"]
        assert err(got, want[:n], dtype) < TOL[dtype], (name, err(got, want[:n], dtype))


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("make", [cfg_mixed, cfg_tiled, cfg_loop_to_the_end])
def test_layer_by_layer_against_the_oracle(tmp_path, device, make):
    """The stream after every layer run (float32): the first one that differs names the mechanism."""
    cfg = make()
    path, cj, W = checkpoint(cfg, tmp_path, seed=2)
    toks = tokens(33, cfg.vocab_size, 4)
    trace = []
    O.forward(cj, W, toks, trace)
    eng = engine(path, device, "float32")
    eng.model.layer_outputs = []
    got = run_schedule(eng, {"a": toks}, [[("a", len(toks))]])["a"]
    assert len(eng.model.layer_outputs) == len(trace) == len(cfg.layer_runs())
    for i, (a, b) in enumerate(zip(eng.model.layer_outputs, trace)):
        assert float((a.cpu().double() - b).abs().max()) < 2e-4 * float(b.abs().max()), i
    assert err(got, oracle_logits(cj, W, toks)) < TOL["float32"]


def test_every_mechanism_shows(tmp_path):
    """The oracle with a pass less, the loop moved, one pass's vector dropped, or any one mechanism off differs by far more
    than the tolerance of these tests."""
    cfg = cfg_mixed()
    _, cj, W = checkpoint(cfg, tmp_path, seed=1, sharpen=_sharp)
    toks = tokens(40, cfg.vocab_size, 1)
    want = oracle_logits(cj, W, toks)

    def differs(cj2=cj, W2=W, by=0.05):
        assert err(oracle_logits(cj2, W2, toks), want) > by

    for change in ({"times": 2}, {"start": 2}, {"stop": 3}):
        c = copy.deepcopy(cj)
        c["loop"].update(change)
        differs(c)
    for t in range(3):
        w = dict(W)
        w["loop.step"] = W["loop.step"].clone()
        w["loop.step"][t] = 0
        differs(W2=w)
    for layer, keys in ((0, ("mix.g", "mlp.router.b")), (1, ("mix.q.b", "mix.k.b", "mlp.router.b"))):
        for k in keys:
            differs(W2={**W, f"l{layer}.{k}": W[f"l{layer}.{k}"] * 0})
    differs(W2={**W, "l0.mix.sink": W["l0.mix.sink"] - 30})
    for k in ("l0.mix.q.norm", "l0.mix.k.norm", "l1.mix.q.norm", "l1.mix.k.norm"):
        differs(W2={**W, k: torch.ones_like(W[k])})
    for path, v in ((("layers", 1, "mixer", "q_temp", "coef"), 0.0), (("layers", 1, "mixer", "q_temp", "every"), 8),
                    (("layers", 0, "mixer", "softcap"), 400.0), (("layers", 0, "mixer", "rot", "scaling"), None),
                    (("layers", 0, "mixer", "rot", "dims"), 8), (("embedding", "scale"), 1.0)):
        c = copy.deepcopy(cj)
        d = c
        for p in path[:-1]:
            d = d[p]
        d[path[-1]] = v
        differs(c, by=0.005)
    assert [i for i, _ in cfg.layer_runs()] == [0, 1, 2, 3, 1, 2, 3, 1, 2, 3, 4, 5]
    assert [(n, t) for n, (_, t) in enumerate(cfg.layer_runs()) if t is not None] == [(1, 0), (4, 1), (7, 2)]


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_mixed_batches_reuse_pages(tmp_path, device, dtype):
    """Unequal requests side by side (portions beside single tokens, a request that pauses), at most three live, in few blocks
    that are freed and used again: every request's logits equal the oracle's for it alone."""
    say("mixed batches", device, dtype)
    cfg = cfg_mixed()
    path, cj, W = checkpoint(cfg, tmp_path, seed=1)
    P = {r: tokens(n, cfg.vocab_size, 10 + i) for i, (r, n) in enumerate([("a", 40), ("b", 23), ("c", 9), ("d", 31), ("e", 1),
                                                                           ("f", 18)])}
    sched = [[("a", 7), ("b", 2)], [("a", 1), ("b", 16), ("c", 3)], [("a", 16), ("c", 1)], [("b", 1), ("c", 1), ("a", 1)],
             [("a", 15), ("b", 4), ("c", 4)],                      # a, b, c end; their pages go back
             [("d", 5), ("e", 1), ("f", 2)], [("d", 1), ("f", 1)], [("f", 15), ("d", 24)], [("d", 1)]]
    eng = engine(path, device, dtype, blocks=7, seqs=3)
    got = run_schedule(eng, P, sched)
    assert len(eng.blocks.free) == 7 and eng.slots is None
    alone = engine(path, device, dtype) if dtype == "bfloat16" else None
    for r, toks in P.items():
        want = oracle_logits(cj, W, toks)
        assert err(got[r], want, dtype) < TOL[dtype], (r, err(got[r], want, dtype))
        if alone is not None:   # the same arithmetic without the batch: closer than the bf16 spread
            ref = run_schedule(alone, {r: toks}, [[(r, len(toks))]])[r]
            assert err(got[r], ref, dtype) < 0.05, (r, err(got[r], ref, dtype))


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("block_size", [16, 64])
def test_block_and_tile_edges(tmp_path, device, block_size):
    """Sharp attention, cuts and decoding at and around the blocks' and the query tiles' edges (float32); a dropped sink, a
    dropped gate or forgotten keys would show."""
    say("edges", device, block_size)
    cfg = cfg_tiled()
    path, cj, W = checkpoint(cfg, tmp_path, seed=5, sharpen=_sharp)
    toks = tokens(140, cfg.vocab_size, 7)
    want = oracle_logits(cj, W, toks)
    for k, v in (("l0.mix.sink", -30.0), ("l3.mix.sink", -30.0)):
        assert err(oracle_logits(cj, {**W, k: W[k] + v}, toks), want) > 50 * TOL["float32"], k
    assert err(oracle_logits(cj, {**W, "l3.mix.g": W["l3.mix.g"] * 0}, toks), want) > 50 * TOL["float32"]
    assert err(oracle_logits(cj, W, toks[64:]), want[64:]) > 50 * TOL["float32"]     # (everything before token 64 forgotten)
    eng = engine(path, device, "float32", block_size=block_size, blocks=12)
    for cuts in ([32, 1, 1, 106], [31, 33, 76], [64, 64, 12], [63, 1, 1, 1, 74], [65, 2, 73], [15, 1, 1, 1, 46, 32, 32, 12],
                 [2] * 70, [127, 1, 1, 11]):
        assert sum(cuts) == len(toks)
        got = run_schedule(eng, {"a": toks}, [[("a", c)] for c in cuts])["a"]
        assert err(got, want) < TOL["float32"], (cuts, err(got, want))


@pytest.mark.gpu
@pytest.mark.parametrize("block_size", [16, 64])
def test_prompt_kernels_bf16(tmp_path, block_size):
    """bfloat16 on the GPU with the shapes the MFMA kernels take: prompts that continue cached context, cut inside tiles and
    blocks, against the oracle and against the same engine run whole."""
    cfg = cfg_tiled()
    path, cj, W = checkpoint(cfg, tmp_path, seed=6)
    toks = tokens(300, cfg.vocab_size, 17)
    want = oracle_logits(cj, W, toks)
    eng = engine(path, "cuda", "bfloat16", block_size=block_size, blocks=512 // block_size)
    whole = run_schedule(eng, {"a": toks}, [[("a", 300)]])["a"]
    assert err(whole, want, "bfloat16") < 0.06, err(whole, want, "bfloat16")
    for cuts in ([70, 230], [33, 31, 1, 235], [40, 1, 1, 1, 257], [17] * 17 + [11], [3, 2, 67, 128, 100], [129, 127, 44]):
        got = run_schedule(eng, {"a": toks}, [[("a", c)] for c in cuts])["a"]
        assert err(got, want, "bfloat16") < 0.06, (cuts, err(got, want, "bfloat16"))
        assert err(got, whole, "bfloat16") < 0.04, (cuts, err(got, whole, "bfloat16"))


@pytest.mark.parametrize("device", DEVICES)
def test_long_decode_and_far_tokens(tmp_path, device):
    """200 tokens decoded one by one after a short prompt, two sequences of different lengths in the batch; attention reaches
    back to the first tokens (the oracle with the first token changed differs at the end)."""
    say("long decode", device)
    cfg = cfg_mixed()
    path, cj, W = checkpoint(cfg, tmp_path, seed=8, sharpen=_sharp)
    a, b = tokens(230, cfg.vocab_size, 20), tokens(120, cfg.vocab_size, 21)
    want_a, want_b = oracle_logits(cj, W, a), oracle_logits(cj, W, b)
    other = oracle_logits(cj, W, [(a[0] + 1) % cfg.vocab_size] + a[1:])
    assert err(other[-5:], want_a[-5:]) > 20 * TOL["float32"]
    eng = engine(path, device, "float32", blocks=30)
    sched = [[("a", 30), ("b", 3)]] + [[("a", 1), ("b", 1)]] * 117 + [[("a", 1)]] * 83
    got = run_schedule(eng, {"a": a, "b": b}, sched)
    assert err(got["a"], want_a) < TOL["float32"] and err(got["b"], want_b) < TOL["float32"]
    if device != "cpu":
        assert eng.runner.graph_replays > 0      # decode steps ran as replayed hipGraphs


def generate(eng, prompts, n, **kw):
    for i, p in enumerate(prompts):
        eng.add_request(f"r{i}", p, SamplingParams(max_tokens=n, ignore_eos=True, **kw))
    outs = {}
    while eng.has_unfinished():
        for o in eng.step():
            if o.finished:
                outs[o.request_id] = list(o.seq.output_ids)
    return outs


@pytest.mark.parametrize("device", DEVICES)
def test_greedy_generation_through_the_scheduler(tmp_path, device):
    """engine.add_request / step(): five requests, three live at a time, greedy; each output token is the oracle's argmax
    (tokens whose top two logits are closer than the tolerance are skipped)."""
    say("generate", device)
    cfg = cfg_mixed()
    path, cj, W = checkpoint(cfg, tmp_path, seed=11)
    eng = engine(path, device, "float32", blocks=12, seqs=3)
    prompts = [tokens(n, cfg.vocab_size, 30 + i) for i, n in enumerate((5, 19, 2, 33, 11))]
    outs = generate(eng, prompts, 12)
    assert len(eng.blocks.free) == 12
    for i, p in enumerate(prompts):
        out = outs[f"r{i}"]
        assert len(out) == 12
        lg = oracle_logits(cj, W, p + out[:-1])[len(p) - 1:]
        for j, t in enumerate(out):
            top = lg[j].topk(2).values
            assert float(lg[j].max() - lg[j][t]) <= 1e-3 * float(lg[j].std()) or float(top[0] - top[1]) < 1e-3, (i, j)


@pytest.mark.parametrize("device", DEVICES)
def test_cached_prefixes_are_adopted(tmp_path, device):
    """The paged planes are all the model keeps, so a prompt that begins like an earlier one takes over its full blocks (also
    those of every pass of the loop) and generates what it would from scratch."""
    cfg = cfg_mixed()
    path, _, _ = checkpoint(cfg, tmp_path, seed=14)
    head = tokens(37, cfg.vocab_size, 60)
    prompts = [head + tokens(5, cfg.vocab_size, 61), head + tokens(9, cfg.vocab_size, 62)]
    fresh = [generate(engine(path, device, "float32"), [p], 8)["r0"] for p in prompts]
    eng = engine(path, device, "float32", prefix=True)
    assert generate(eng, prompts[:1], 8)["r0"] == fresh[0]
    seq = eng.add_request("second", prompts[1], SamplingParams(max_tokens=8, ignore_eos=True))
    eng.step()
    assert eng.blocks.hit_tokens == 32      # two full blocks of 16
    while eng.has_unfinished():
        eng.step()
    assert list(seq.output_ids) == fresh[1]


@pytest.mark.gpu
def test_pipelined_decode_takes_the_previous_token_from_the_device(tmp_path):
    """Pipelined decode: a step's input token is the sample the step before left on the device; the outputs equal those of
    the engine that waits for every step."""
    cfg = cfg_mixed()
    path, _, _ = checkpoint(cfg, tmp_path, seed=12)
    prompts = [tokens(n, cfg.vocab_size, 40 + i) for i, n in enumerate((7, 21, 3))]
    outs = [generate(engine(path, "cuda", "float32", blocks=12, seqs=3, pipeline=pipe), prompts, 20) for pipe in (False, True)]
    assert outs[0] == outs[1] and all(len(v) == 20 for v in outs[0].values())


def test_preempted_requests_start_over(tmp_path):
    """A pool too small for the decoded tails: a sequence is preempted, its pages are taken by another, and its recomputation
    gives the same tokens as in a pool with room."""
    cfg = cfg_mixed()
    path, _, _ = checkpoint(cfg, tmp_path, seed=13)
    prompts = [tokens(n, cfg.vocab_size, 50 + i) for i, n in enumerate((14, 17, 12))]
    outs = {}
    for blocks in (5, 24):
        eng = engine(path, "cpu", "float32", blocks=blocks, seqs=3)
        outs[blocks] = generate(eng, prompts, 30)
        assert len(eng.blocks.free) == blocks
    assert outs[5] == outs[24] and all(len(v) == 30 for v in outs[5].values())


def test_config_reader_rejects_unknown_keys_and_roundtrips():
    for make in ALL:
        cfg = make()
        assert C.from_config_json(C.bekedra_to_config(cfg), cfg.name) == cfg
    cj = C.bekedra_to_config(cfg_mixed())

    def bad(change):
        c = copy.deepcopy(cj)
        change(c)
        with pytest.raises(ValueError):
            C.from_config_json(c, "x")

    bad(lambda c: c["layers"][1]["mixer"].update(window=8))
    bad(lambda c: c["layers"][0]["mixer"]["rot"]["scaling"].update(extra=1))
    bad(lambda c: c["layers"][0]["mixer"]["rot"].update(dims=16))
    bad(lambda c: c["layers"][1]["mixer"].update(kv_heads=4))
    bad(lambda c: c["layers"][1]["mixer"].update(vdim=4))
    bad(lambda c: c["layers"][0]["mlp"]["router"].update(top=8))
    bad(lambda c: c["layers"][0]["mlp"].update(kind="dense"))
    bad(lambda c: c["loop"].update(stop=99))
    bad(lambda c: c.update(streams=2))
    bad(lambda c: c["layers"][0].update(type="delta"))
    assert C.resolve("tiny-bekedra").family == "bekedra"
    kv = C.resolve("small-bekedra")
    assert kv.kv_bytes_per_token() == 2 * (4 * 128 * 2 + 4) + 2 * (2 * 4 * 128 * 2)


def test_registered_model_by_name_and_checkpoint_tensors(tmp_path):
    """The registry name runs with random weights as every other modelName does (the command line's path), and equals the
    oracle; a checkpoint with a tensor too many or too few is refused."""
    from safetensors.torch import load_file, save_file

    from symmetry_amd.models.weights import random_weights

    c = C.resolve("tiny-bekedra")
    eng = LLMEngine(EngineConfig(model="tiny-bekedra", weights="random", dtype="float32", device="cpu", max_num_seqs=2,
                                 block_size=16, num_kv_blocks=9, max_model_len=128, use_graphs=False,
                                 enable_prefix_caching=False, pipeline=False, seed=3))
    W = {k: v.to(BF16) for k, v in random_weights(c, seed=3).tensors.items()}
    toks = tokens(50, c.vocab_size, 2)
    got = run_schedule(eng, {"a": toks}, [[("a", 31)], [("a", 19)]])["a"]
    assert err(got, oracle_logits(C.bekedra_to_config(c), W, toks)) < TOL["float32"]
    path, _, _ = checkpoint(cfg_mixed(), tmp_path, seed=4)
    f = os.path.join(path, "model.safetensors")
    t = load_file(f)
    t["l1.mix.v"] = torch.ones(4)
    save_file(t, f)
    with pytest.raises(ValueError):
        engine(path, "cpu", "float32")
    del t["l1.mix.v"], t["loop.step"]
    save_file(t, f)
    with pytest.raises(ValueError):
        engine(path, "cpu", "float32")


# ---- mechanisms alone: op against oracle function ---------------------------------------------------------------
def _dev(device, *ts):
    return [t.to(device) if torch.is_tensor(t) else t for t in ts]


def _paged(n, BS, seed):
    """A block table over shuffled blocks (block 0 stays unused), positions and cache rows of n tokens."""
    NB = n // BS + 3
    bt = (torch.randperm(NB - 1, generator=torch.Generator().manual_seed(seed))[None] + 1).int()
    pos = torch.arange(n, dtype=torch.int32)
    slots = (bt[0][(pos // BS).long()] * BS + pos % BS).int()
    return NB, bt, pos, slots


def close(a, b, tol):
    d = float((a.cpu().double() - b.double()).abs().max())
    assert d < tol * max(1.0, float(b.double().abs().max())), d


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("shape", [(6, 2, 10, 14, 3), (4, 4, 16, 8, 8), (3, 1, 96, 64, 32), (2, 2, 200, 256, 0), (8, 4, 64, 40, 5)])
def test_head_norms_and_rotation_into_the_cache(device, dtype, shape):
    """Per-head norms, then the half-layout rotation at far positions, q out and k / v into shuffled cache rows; a row without
    a slot writes nothing."""
    H, G, dk, dv, pairs = shape
    say("op qk_norm_cache rotary", device, dtype, shape)
    torch.manual_seed(dk)
    n, BS = 21, 16
    z = torch.randn(n, H * dk + G * (dk + dv) + 8).to(dtype)
    wq, wk = torch.rand(dk) + 0.5, torch.rand(dk) + 0.5
    rot = {"dims": 2 * pairs, "base": 300.0, "scaling": {"factor": 4.0, "low": 1.0, "high": 4.0, "original": 100}}
    NB, _, _, slots = _paged(n, BS, 1)
    pos = (torch.arange(n) * 97 % 1500).int()
    slots[5] = -1
    rope = None
    if pairs:
        t = ops.rope_table(1500, 2 * pairs, 300.0, {"rope_type": "llama3", "factor": 4.0, "low_freq_factor": 1.0,
                                                    "high_freq_factor": 4.0, "original_max_position_embeddings": 100})
        rope = t.view(1500, 2, pairs).transpose(1, 2).contiguous()
    q, kc, vc = torch.zeros(n, H, dk), torch.zeros(NB, BS, G, dk), torch.zeros(NB, BS, G, dv)
    q, kc, vc = q.to(dtype), kc.to(dtype), vc.to(dtype)
    zd, wqd, wkd, sd, qd, kd, vd, rd, pd = _dev(device, z, wq, wk, slots, q, kc, vc, rope, pos)
    ops.qk_norm_cache(zd[:, :H * dk + G * (dk + dv)], H, G, dk, dv, wqd, wkd, None, 1e-5, sd, qd, kd, vd, rope=rd, positions=pd)
    zf = z.double()
    wq_, wk_ = O.rms_norm(zf[:, :H * dk].view(n, H, dk), wq.double(), 1e-5), O.rms_norm(
        zf[:, H * dk:(H + G) * dk].view(n, G, dk), wk.double(), 1e-5)
    if pairs:
        wq_, wk_ = O.rotate_half(wq_, pos, rot), O.rotate_half(wk_, pos, rot)
    tol = 2e-5 if dtype == F32 else 6e-3
    close(qd, wq_, tol)
    keep = slots >= 0
    close(kd.cpu().view(-1, G, dk)[slots[keep].long()], wk_[keep], tol)
    close(vd.cpu().view(-1, G, dv)[slots[keep].long()], zf[:, (H + G) * dk:(H + G) * dk + G * dv].view(n, G, dv)[keep], 1e-7)
    used = torch.zeros(NB * BS, dtype=torch.bool)
    used[slots[keep].long()] = True
    assert float(kd.cpu().view(-1, G * dk)[~used].float().abs().max()) == 0


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("shape", [(6, 2, 10), (4, 4, 16), (3, 1, 64), (16, 4, 128), (2, 2, 33)])
def test_keys_that_are_values(device, dtype, shape):
    """Biases, norms over whole projections, query temperature at its steps, one cached plane: prompt rows and single rows give
    the oracle's attention; a far key that one query looks hard at, at block borders and at position 0."""
    H, G, D = shape
    say("op qk_row_norm_cache + attention", device, dtype, shape)
    torch.manual_seed(D)
    n, BS, scale = 150, 16, 0.5 * D ** -0.5
    m = {"heads": H, "kv_heads": G, "dim": D, "scale": scale, "q_temp": {"coef": 0.7, "every": 10}}
    tol = 3e-5 if dtype == F32 else 3e-2
    z = torch.randn(n, (H + G) * D)
    bias, wq, wk = torch.randn((H + G) * D) * 0.3, torch.rand(H * D) + 0.5, torch.rand(G * D) + 0.5
    for target in (0, 15, 16, 63, 64, 100, 148):
        z2 = z.clone()      # the last query of every head points at the target's key, and that key stands out
        z2[target, H * D:] *= 3.0
        z2[149, :H * D] = (6.0 * z2[target, H * D:].view(G, D)).repeat_interleave(H // G, 0).reshape(-1)
        z2 = z2.to(dtype)
        zb = z2.double() + bias.double()
        q, k = zb[:, :H * D], zb[:, H * D:]
        qn = O.rms_norm(q, wq.double(), 1e-5).view(n, H, D) * O.query_temperature(torch.arange(n), 0.7, 10)[:, None, None]
        s = O.causal_scores(qn, O.rms_norm(k, wk.double(), 1e-5).view(n, G, D), scale)
        want = O.mix_values(O.causal_softmax(s), k.view(n, G, D), H)
        blind = s.clone()
        blind[:, :, target] = -1e9
        assert float((O.mix_values(O.causal_softmax(blind), k.view(n, G, D), H)[149] - want[149]).abs().max()) > 0.3
        NB, bt, pos, slots = _paged(n, BS, 2)
        q_out = torch.zeros(n, H, D, dtype=dtype)
        kc, ks = torch.zeros(NB, BS, G, D, dtype=dtype), torch.zeros(NB, BS)
        out, rs, cu = torch.empty(n, H, D, dtype=dtype), torch.zeros(n, dtype=torch.int32), torch.tensor([0, n]).int()
        tiles = torch.tensor([[0, r] for r in range(0, n, 64)] + [[0, 1 << 20]]).int()
        zd, bd, wqd, wkd, bt, pos, slots, q_out, kc, ks, out, rs, cu, tiles = _dev(
            device, z2, bias, wq, wk, bt, pos, slots, q_out, kc, ks, out, rs, cu, tiles)
        ops.qk_row_norm_cache(zd, bd, H, G, D, wqd, wkd, 1e-5, 0.7, 10, pos, slots, q_out, kc, ks)
        impl = ops.window_attn(q_out, kc, kc, bt, rs, pos, CAUSAL, scale, None, out, tiles, cu, key_scale=ks)
        assert device == "cpu" or impl == (2 if dtype == BF16 and D in (64, 128) else impl)
        close(out.reshape(n, -1), want, tol)
        one = torch.empty(1, H, D, dtype=dtype, device=device)
        ops.window_attn(q_out[149:], kc, kc, bt, rs[:1], pos[149:], CAUSAL, scale, None, one, key_scale=ks)
        close(one.reshape(1, -1), want[149:], tol)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("cap", [2.0, 30.0, 500.0])
@pytest.mark.parametrize("shape", [(4, 4, 96, 96), (4, 2, 32, 32), (6, 2, 12, 20), (3, 1, 80, 80)])
def test_capped_scores_sink_and_column_gate(device, dtype, cap, shape):
    """Soft cap below, above and far above the scores' size, sink, element-wise gate read from a column range; prompt rows that
    continue a cached context and single rows; keys at borders that one query looks hard at; a sink that takes everything."""
    H, G, D, P = shape
    say("op window_attn softcap", device, dtype, cap, shape)
    torch.manual_seed(D)
    n, BS, first = 150, 16, 37
    tol = 3e-5 if dtype == F32 else 2e-2
    NB, bt, pos, slots = _paged(n, BS, 3)
    k, v = torch.randn(n, G, D).to(dtype), torch.randn(n, G, P).to(dtype)
    kc, vc = torch.zeros(NB, BS, G, D, dtype=dtype), torch.zeros(NB, BS, G, P, dtype=dtype)
    kc.view(-1, G, D)[slots.long()], vc.view(-1, G, P)[slots.long()] = k, v
    gate = torch.randn(n, H * P + 8).to(dtype)
    sink = torch.randn(H)
    sink[0] = 2.0 * min(cap, 40.0)      # head 0: nothing outweighs it by much
    for target in (0, 15, 16, 63, 64, 127, 149):
        q = torch.randn(n, H, D)
        q[149] = 4.0 * k[target].float().repeat_interleave(H // G, 0)
        q = q.to(dtype)
        s = O.soft_cap(O.causal_scores(q.double(), k.double(), 0.3), cap)
        want = O.mix_values(O.causal_softmax(s, sink.double()), v.double(), H) * torch.sigmoid(gate[:, :H * P].double())
        rows = slice(first, n)          # the rows before are cached context
        T = n - first
        rs, cu = torch.zeros(T, dtype=torch.int32), torch.tensor([0, T]).int()
        tiles = torch.tensor([[0, r] for r in range(0, T, 64)] + [[0, 1 << 20]]).int()
        out = torch.empty(T, H, P, dtype=dtype)
        qd, gd, kcd, vcd, btd, rsd, posd, sd, out, cud, td = _dev(device, q, gate, kc, vc, bt, rs, pos, sink, out, cu, tiles)
        ops.window_attn(qd[rows].contiguous(), kcd, vcd, btd, rsd, posd[rows].contiguous(), CAUSAL, 0.3, gd[rows, :H * P], out,
                        td, cud, sink=sd, softcap=cap)
        close(out.reshape(T, -1), want[rows], tol)
        one = torch.empty(1, H, P, dtype=dtype, device=device)
        ops.window_attn(qd[149:], kcd, vcd, btd, rsd[:1], posd[149:], CAUSAL, 0.3, gd[149:, :H * P], one, sink=sd, softcap=cap)
        close(one.reshape(1, -1), want[149:], tol)
    nosink = O.mix_values(O.causal_softmax(s), v.double(), H) * torch.sigmoid(gate[:, :H * P].double())
    uncapped = O.mix_values(O.causal_softmax(O.causal_scores(q.double(), k.double(), 0.3), sink.double()), v.double(), H)
    assert float((nosink - want).abs().max()) > 0.2
    if cap < 10:
        assert float((uncapped * torch.sigmoid(gate[:, :H * P].double()) - want).abs().max()) > 0.2


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", [F32, BF16])
@pytest.mark.parametrize("T", [1, 5, 16, 17, 130])
@pytest.mark.parametrize("shape", [(32, 3, 1, 24), (64, 10, 3, 64), (96, 40, 40, 32), (72, 20, 5, 18), (160, 100, 7, 96)])
def test_router_and_experts(device, dtype, T, shape):
    """The biased choice, softmax over the chosen logits, segment bounds and places, gathered expert products with the squared
    ReLU, and the weighted sum into the stream with the next norm -- against the oracle token by token; an expert that nobody
    chooses and one that everybody does."""
    d, E, k, ff = shape
    say("op route / experts", device, dtype, T, shape)
    torch.manual_seed(d + T)
    h = torch.randn(T, d).to(dtype)
    W = {"m.router": (3.0 * torch.randn(E, d) * d ** -0.5).to(dtype), "m.router.b": torch.randn(E)}
    if 1 < k < E:
        W["m.router.b"][E - 1], W["m.router.b"][0] = -1e3, 1e3
    for e in range(E):
        W[f"m.e{e}.up"] = (torch.randn(ff, d) * d ** -0.5).to(dtype)
        W[f"m.e{e}.down"] = (torch.randn(d, ff) * ff ** -0.5).to(dtype)
    Wd = {n: v.double() for n, v in W.items()}
    ids_w, wts_w = O.route(Wd, "m.", k, h.double())
    i32 = torch.int32
    ids, w = torch.zeros(T * k, dtype=i32), torch.zeros(T * k)
    off, dst, src = torch.zeros(E + 1, dtype=i32), torch.zeros(T * k, dtype=i32), torch.zeros(T * k, dtype=i32)
    hd, Wr, br, ids, w, off, dst, src = _dev(device, h, W["m.router"], W["m.router.b"], ids, w, off, dst, src)
    ops.route_topk(hd, Wr, br, k, ids, w, off, dst, src)
    z = (h.double() @ Wd["m.router"].T + Wd["m.router.b"]).sort(-1, descending=True).values
    sure = torch.ones(T, dtype=torch.bool) if k == E else (z[:, k - 1] - z[:, k]) > 1e-4
    got, want = ids.cpu().view(T, k).long(), ids_w
    assert torch.equal(got[sure].sort(-1).values, want[sure].sort(-1).values)
    for t in range(T):
        if sure[t]:
            ww = {int(e): float(x) for e, x in zip(ids_w[t], wts_w[t])}
            assert all(abs(float(w[t * k + j]) - ww[int(got[t, j])]) < 1e-5 for j in range(k)), t
    o, places = off.cpu().long(), dst.cpu().long()
    assert int(o[0]) == 0 and int(o[E]) == T * k and sorted(places.tolist()) == list(range(T * k))
    flat = got.reshape(-1)
    assert torch.all(places >= o[flat]) and torch.all(places < o[flat + 1])
    assert torch.equal(src.cpu().long()[places], torch.arange(T * k) // k)
    if 1 < k < E:
        assert int(o[1]) == T and int(o[E]) == int(o[E - 1])
    up = torch.stack([W[f"m.e{e}.up"] for e in range(E)]).to(device)
    down = torch.stack([W[f"m.e{e}.down"] for e in range(E)]).to(device)
    act, y = torch.empty(T * k, ff, dtype=dtype, device=device), torch.empty(T * k, d, dtype=dtype, device=device)
    ops.expert_linear(hd, src, up, off, act, relu2=True)
    ops.expert_linear(act, None, down, off, y)
    x, a, bias, wn = torch.randn(T, d), torch.randn(T, d).to(dtype), torch.randn(d), torch.rand(d) + 0.5
    out = torch.empty(T, d, dtype=dtype)
    xd, ad, bd, wnd, out = _dev(device, x.clone(), a, bias, wn, out)
    ops.residual_routed_norm(xd, ad, y, dst, w, k, bd, wnd, 1e-5, out)
    ff_w = torch.zeros(T, d, dtype=F64)
    for t in range(T):
        for j in range(k):      # (the op's own choice, so that a tie that rounding breaks the other way is no error)
            e = int(got[t, j])
            ff_w[t] += float(w[t * k + j]) * O.expert(Wd, f"m.e{e}.", h[t].double())
    new = x.double() + a.double() + ff_w + bias.double()
    close(xd, new, 2e-5 if dtype == F32 else 2e-2)
    close(out, O.rms_norm(new, wn.double(), 1e-5), 2e-5 if dtype == F32 else 3e-2)
    x2 = xd.clone()
    ops.residual_routed_norm(xd, None, None, None, None, 0, None)
    assert torch.equal(x2, xd)


@pytest.mark.gpu
@pytest.mark.parametrize("R", [40, 700, 3000])
@pytest.mark.parametrize("shape", [(4, 128, 192), (7, 200, 64), (3, 260, 320)])
def test_expert_product_forms_agree(R, shape):
    """Every form of the expert product (all shapes, weight stream, both tiles) on uneven segments, one of them empty, with
    gathered rows and without: the product of bf16 values, whatever the form."""
    E, N, K = shape
    say("op expert_linear forms", R, shape)
    from symmetry_amd.ops import _native

    torch.manual_seed(N)
    cuts = sorted(torch.randint(0, R + 1, (E - 2,)).tolist())
    off = torch.tensor([0, 0] + cuts + [R]).int()
    x, W = torch.randn(R // 2 + 1, K).to(BF16), (torch.randn(E, N, K) * K ** -0.5).to(BF16)
    src = torch.randint(0, x.shape[0], (R,)).int()
    want = torch.zeros(R, N)
    for e in range(E):
        a, b = int(off[e]), int(off[e + 1])
        want[a:b] = x[src[a:b].long()].float() @ W[e].float().t()
    for impl in (0, 1, 2, 3, -1):
        for relu2 in (True, False):
            y = torch.full((R, N), 7.0, dtype=BF16, device="cuda")
            _native.hybrid_ops().expert_linear(x.cuda(), src.cuda(), W.cuda(), off.cuda(), y, relu2, impl)
            close(y.float(), torch.relu(want) ** 2 if relu2 else want, 6e-3)
        xs = x[src.long()].cuda()
        y2 = torch.full((R, N), 7.0, dtype=BF16, device="cuda")
        _native.hybrid_ops().expert_linear(xs, None, W.cuda(), off.cuda(), y2, False, impl)
        close(y2.float(), want, 6e-3)


@pytest.mark.gpu
@pytest.mark.parametrize("D", [32, 48, 64, 80, 96, 112, 128])
@pytest.mark.parametrize("BS", [16, 24, 64, 128])
def test_prompt_kernel_on_unequal_runs(D, BS):
    """The causal prompt kernel on a batch of unequal runs (one row, two rows, runs around 64 and 128, cached context before
    them) in blocks smaller and larger than a key tile: against the oracle, sequence by sequence."""
    say("op prompt kernel", D, BS)
    torch.manual_seed(D)
    H, G = 4, 2
    lens, ctx = [1, 2, 63, 64, 130, 129], [0, 70, 3, 64, 0, 200]
    S = len(lens)
    mb = max(-(-(a + b) // BS) for a, b in zip(lens, ctx))
    bt = (torch.randperm(S * mb) + 1).view(S, mb).int()
    k, v = torch.randn(S * mb + 1, BS, G, D).to(BF16), torch.randn(S * mb + 1, BS, G, D).to(BF16)
    T = sum(lens)
    q = (2.0 * torch.randn(T, H, D)).to(BF16)
    pos = torch.cat([torch.arange(c, c + n) for c, n in zip(ctx, lens)]).int()
    rs = torch.repeat_interleave(torch.arange(S), torch.tensor(lens)).int()
    cu = torch.tensor([0] + torch.tensor(lens).cumsum(0).tolist()).int()
    tiles = torch.tensor([[i, r] for i, n in enumerate(lens) for r in range(0, n, 64)] + [[0, 1 << 20]]).int()
    sink = torch.randn(H)
    for cap, same, ks in ((0.0, False, None), (0.0, True, torch.rand(S * mb + 1, BS) + 0.3), (5.0, False, None)):
        vv = k if same else v
        out = torch.full((T, H, D), 9.0, dtype=BF16, device="cuda")
        kd = k.cuda()
        impl = ops.window_attn(q.cuda(), kd, kd if same else v.cuda(), bt.cuda(), rs.cuda(), pos.cuda(), CAUSAL, D ** -0.5,
                               None, out, tiles.cuda(), cu.cuda(), sink=sink.cuda(), softcap=cap,
                               key_scale=None if ks is None else ks.cuda())
        assert impl == 2
        for i, (n, c) in enumerate(zip(lens, ctx)):
            idx = torch.arange(c + n)
            K = k[bt[i][idx // BS].long(), idx % BS].double()
            V = vv[bt[i][idx // BS].long(), idx % BS].double()
            full = torch.zeros(c + n, H, D, dtype=F64)
            full[c:] = q[int(cu[i]):int(cu[i]) + n].double()
            s = O.causal_scores(full, K, D ** -0.5)
            if ks is not None:
                s = s * ks[bt[i][idx // BS].long(), idx % BS].double()
            if cap:
                s = O.soft_cap(s, cap)
            want = O.mix_values(O.causal_softmax(s, sink.double()), V, H)[c:]
            close(out[int(cu[i]):int(cu[i]) + n].reshape(n, -1), want, 1.5e-2)


@pytest.mark.gpu
@pytest.mark.parametrize("D", [32, 48, 64, 80, 96, 112, 128])
@pytest.mark.parametrize("keys", [None, 32, 64, 256, 4096])
def test_key_ranges_of_single_rows(D, keys):
    """Decode attention by key ranges: contexts of one key up to many ranges, last ranges of one key, in blocks of 16, 24 and
    64, one to eight query heads per key head; against the oracle, twice through the same workspace (the arrival counters are
    back at zero)."""
    say("op split attention", D, keys)
    torch.manual_seed(D)
    for H, G, BS, cap, same, per_col in ((8, 4, 64, 6.0, False, True), (4, 4, 16, 0.0, True, False), (8, 1, 24, 80.0, False, False)):
        ctx = [1, 2, 31, 32, 33, 64, 65, 128, 129, 300, 1025]
        T, mb = len(ctx), -(-max(ctx) // BS)
        bt = (torch.randperm(T * mb) + 1).view(T, mb).int()
        k, v = torch.randn(T * mb + 1, BS, G, D).to(BF16), torch.randn(T * mb + 1, BS, G, D).to(BF16)
        ks = torch.rand(T * mb + 1, BS) + 0.3 if same else None
        q, sink = (2.0 * torch.randn(T, H, D)).to(BF16), torch.randn(H)
        gate = torch.randn(T, H * D if per_col else H).to(BF16)
        pk, parts = ops.window_attn_split(T, G, mb * BS)
        if keys:
            pk, parts = keys, -(-mb * BS // keys)
        ws = (torch.full((T, H, parts, D), float("nan"), device="cuda"), torch.full((T, H, parts, 2), float("nan"), device="cuda"),
              torch.zeros(T * G, dtype=torch.int32, device="cuda"), pk)
        kd = k.cuda()
        args = [q.cuda(), kd, kd if same else v.cuda(), bt.cuda(), torch.arange(T).int().cuda(),
                (torch.tensor(ctx) - 1).int().cuda()]
        for _ in range(2):
            out = torch.full((T, H, D), 9.0, dtype=BF16, device="cuda")
            impl = ops.window_attn(*args, CAUSAL, D ** -0.5, gate.cuda(), out, sink=sink.cuda(), softcap=cap,
                                   key_scale=None if ks is None else ks.cuda(), split=ws)
            assert impl == (3 if parts <= 64 else 0)
            assert int(ws[2].abs().max()) == 0
            for t, n in enumerate(ctx):
                idx = torch.arange(n)
                at = bt[t][idx // BS].long(), idx % BS
                K, V = k[at].double(), (k if same else v)[at].double()
                full = torch.zeros(n, H, D, dtype=F64)
                full[-1] = q[t].double()
                s = O.causal_scores(full, K, D ** -0.5)
                if ks is not None:
                    s = s * ks[at].double()
                if cap:
                    s = O.soft_cap(s, cap)
                want = O.mix_values(O.causal_softmax(s, sink.double()), V, H)[-1].view(H, D)
                close(out[t], want * torch.sigmoid(gate[t].double()).view(H, -1), 1.5e-2)
