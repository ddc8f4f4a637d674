"""Beletar through the engine and op by op, against the plain oracle in tests/beletar_oracle.py.

Every test builds its own small configuration and random weights (sizes all different from one another and from any
shipped checkpoint), writes them as a checkpoint, loads that through the engine, and compares with the oracle.  The CPU
runs use the torch reference ops, the ``gpu`` ones the HIP kernels; float32 comparisons are tight (rounding only),
bfloat16 ones use the spread that bf16 rounding gives.  A dictated step goes through LLMEngine.replay_step, i.e. the
scheduler, the block / slot managers, the runner's packed metadata (and decode hipGraphs on the GPU) and model.forward.
"""
from __future__ import annotations

import copy
import dataclasses
import os
import sys

import pytest
import torch

sys.path.insert(0, os.path.dirname(os.path.abspath(__file__)))
import beletar_oracle as O  # noqa: E402

from symmetry_amd import ops  # noqa: E402
from symmetry_amd.engine.llm_engine import EngineConfig, LLMEngine  # noqa: E402
from symmetry_amd.engine.sequence import SamplingParams  # noqa: E402
from symmetry_amd.models import config as C  # noqa: E402
from symmetry_amd.models.weights import beletar_random_weights, save_beletar_checkpoint  # noqa: E402

DEVICES = ["cpu", pytest.param("cuda", marks=pytest.mark.gpu)]
F64 = torch.float64


def say(*a):
    print(*a, flush=True)


# ---- configurations ---------------------------------------------------------------------------------------------
def head_delta(heads=4, kv=2, dim=10, vdim=14, conv=3):
    return C.DeltaSpec(heads, kv, dim, vdim, conv)


def chan_delta(heads=3, kv=1, dim=7, vdim=5, conv=4, ra=6, rg=9):
    return C.DeltaSpec(heads, kv, dim, vdim, conv, True, ra, rg)


def latent(heads=5, dim=12, rot=8, vdim=9, rank=22, scale=0.3, base=300.0, dims=None, scaling=(3.0, 40.0, 4.0, 0.5)):
    return C.LatentMixerSpec(heads, dim, rot, vdim, rank, 0, base, dims or rot, scale, head_gate=True, sink=True,
                             rot_scaling=scaling)


def lay(kind, mixer, ff=None):
    return C.BeletarLayer(kind, mixer, C.SiluGluSpec(ff) if ff else None)


def cfg_mixed(width=40, vocab=67):
    """Every branch once: both kinds of delta layer with shared and with own query / key heads, latent layers inside and
    outside the loop (so every pass has a plane of its own), layers without feed-forward (one of them the loop's last),
    1 / 2 / 3 / 4 / 6 taps, all head sizes different from one another, frequency blending with and without, part of the
    rotated dims turning."""
    layers = (
        lay("latent_attention", latent(), 36),
        lay("delta", head_delta(), 20),
        lay("channel_delta", chan_delta(), 28),
        lay("latent_attention", latent(heads=2, dim=6, rot=4, vdim=16, rank=13, scale=0.5, scaling=None)),
        lay("channel_delta", chan_delta(heads=2, kv=2, dim=16, vdim=12, conv=6, ra=3, rg=4), 24),
        lay("delta", head_delta(heads=2, kv=2, dim=21, vdim=6, conv=2)),
        lay("delta", head_delta(heads=3, kv=3, dim=5, vdim=33, conv=1), 16),
    )
    return C.BeletarConfig(name="t-mixed", vocab_size=vocab, hidden_size=width, layers=layers, loop=C.LoopSpec(1, 4, 3),
                           embed_scale=3.0, norm_eps=1e-5)


def cfg_tiled(width=64, vocab=97):
    """Sizes that the tiled attention kernel and whole matrix tiles take: cache rows of 64 and 96, key channels 16 / 32 /
    64, the loop over all layers but the last."""
    layers = (
        lay("delta", head_delta(heads=4, kv=2, dim=32, vdim=48, conv=4), 96),
        lay("latent_attention", latent(heads=6, dim=24, rot=16, vdim=32, rank=48, scale=0.2, base=1000.0,
                                       scaling=(8.0, 100.0, 16.0, 1.0)), 64),
        lay("channel_delta", chan_delta(heads=2, kv=1, dim=64, vdim=80, conv=4, ra=16, rg=8), 96),
        lay("channel_delta", chan_delta(heads=8, kv=4, dim=16, vdim=16, conv=3, ra=8, rg=8), 32),
        lay("latent_attention", latent(heads=3, dim=40, rot=32, vdim=20, rank=64, scale=0.15, base=50.0, scaling=None), 64),
    )
    return C.BeletarConfig(name="t-tiled", vocab_size=vocab, hidden_size=width, layers=layers, loop=C.LoopSpec(0, 4, 2),
                           embed_scale=6.0, norm_eps=1e-6)


def cfg_plain(width=24, vocab=50):
    """The values at which mechanisms vanish: one pass, one head, one tap, embedding scale one, no frequency blending."""
    layers = (lay("delta", head_delta(heads=1, kv=1, dim=8, vdim=8, conv=1), 16),
              lay("latent_attention", latent(heads=1, dim=8, rot=2, vdim=4, rank=8, scale=1.0, scaling=None)),
              lay("channel_delta", chan_delta(heads=1, kv=1, dim=4, vdim=4, conv=1, ra=1, rg=1), 8))
    return C.BeletarConfig(name="t-plain", vocab_size=vocab, hidden_size=width, layers=layers, loop=C.LoopSpec(1, 2, 1),
                           embed_scale=1.0, norm_eps=1e-5)


def cfg_noloop():
    return dataclasses.replace(cfg_plain(width=28), name="t-noloop", loop=None)


def cfg_loop_to_the_end():
    """The loop covers the last layer, so the output norm follows a pass."""
    return dataclasses.replace(cfg_plain(width=20), name="t-loopend", loop=C.LoopSpec(1, 3, 4), embed_scale=0.7)


ALL = [cfg_mixed, cfg_tiled, cfg_plain, cfg_noloop, cfg_loop_to_the_end]


def checkpoint(cfg, tmp_path, seed=0, sharpen=None):
    w = beletar_random_weights(cfg, seed=seed)
    if sharpen:
        sharpen(w.tensors)
    path = str(tmp_path / f"{cfg.name}-{seed}")
    save_beletar_checkpoint(w, path)
    return path, C.beletar_to_config(cfg), {k: v.to(torch.bfloat16) for k, v in w.tensors.items()}


def engine(path, device, dtype, blocks=24, seqs=4, block_size=16, graphs=True, pipeline=False):
    return LLMEngine(EngineConfig(model="t", weights=path, dtype=dtype, device=device, max_num_seqs=seqs,
                                  block_size=block_size, num_kv_blocks=blocks + 1, max_model_len=blocks * block_size,
                                  max_num_batched_tokens=8192, use_graphs=graphs, enable_prefix_caching=False,
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
    """The worst row's distance in units of the logits' spread; in bfloat16 the distance that nine rows in ten keep (heads
    of a few entries whose output happens to be small are normed up with their rounding, and such rows stand out)."""
    d = (a.double() - b.double())
    d = d - d.mean(-1, keepdim=True)
    e = d.pow(2).mean(-1).sqrt() / b.double().std(-1).clamp_min(1e-6)
    return float(e.max() if dtype == "float32" else e.quantile(0.9))


TOL = {"float32": 2e-4, "bfloat16": 0.2}    # bf16: a lost mechanism gives errors near 1 in most rows


def oracle_logits(cj, W, toks):
    return O.forward(cj, W, toks).float()


def _sharp(t):
    """Attention that looks hard at single keys and states that forget slowly: a lost key, a lost state or a dropped sink
    moves the logits by far more than the tolerance."""
    for k in t:
        if k.endswith("mix.q") and k.replace("mix.q", "mix.dkv") in t:
            t[k] = t[k] * 4.0
        if k.endswith("dt_bias"):
            t[k] = t[k] - 3.0
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
@pytest.mark.parametrize("make", [cfg_mixed, cfg_loop_to_the_end])
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


def test_loop_passes_show(tmp_path):
    """The oracle with a pass less, with the loop moved, or without the added embedding output differs by far more than the
    tolerance of these tests."""
    cfg = cfg_mixed()
    _, cj, W = checkpoint(cfg, tmp_path, seed=1)
    toks = tokens(30, cfg.vocab_size, 1)
    want = oracle_logits(cj, W, toks)
    for change in ({"times": 2}, {"start": 2}, {"stop": 3}):
        cj2 = copy.deepcopy(cj)
        cj2["loop"].update(change)
        assert err(oracle_logits(cj2, W, toks), want) > 0.3, change
    runs = O.layer_runs
    try:
        O.layer_runs = lambda c: [(i, False) for i, _ in runs(c)]
        assert err(oracle_logits(cj, W, toks), want) > 0.3
    finally:
        O.layer_runs = runs
    assert [i for i, _ in cfg.layer_runs()] == [0, 1, 2, 3, 1, 2, 3, 1, 2, 3, 4, 5, 6]
    assert [n for n, (_, again) in enumerate(cfg.layer_runs()) if again] == [4, 7]


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_mixed_batches_reuse_pages_and_slots(tmp_path, device, dtype):
    """Unequal requests side by side (portions beside single tokens, a request that pauses), in a pool of three slots
    and few blocks that are freed and used again: every request's logits equal the oracle's for it alone."""
    say("mixed batches", device, dtype)
    cfg = cfg_mixed()
    path, cj, W = checkpoint(cfg, tmp_path, seed=1)
    P = {r: tokens(n, cfg.vocab_size, 10 + i) for i, (r, n) in enumerate([("a", 40), ("b", 23), ("c", 9), ("d", 31), ("e", 1),
                                                                           ("f", 18)])}
    sched = [[("a", 7), ("b", 2)], [("a", 1), ("b", 16), ("c", 3)], [("a", 16), ("c", 1)], [("b", 1), ("c", 1), ("a", 1)],
             [("a", 15), ("b", 4), ("c", 4)],                      # a, b, c end; their pages and slots go back
             [("d", 5), ("e", 1), ("f", 2)], [("d", 1), ("f", 1)], [("f", 15), ("d", 24)], [("d", 1)]]
    eng = engine(path, device, dtype, blocks=7, seqs=3)
    got = run_schedule(eng, P, sched)
    assert len(eng.blocks.free) == 7 and eng.slots.num_free == 3
    alone = engine(path, device, dtype) if dtype == "bfloat16" else None
    for r, toks in P.items():
        want = oracle_logits(cj, W, toks)
        assert err(got[r], want, dtype) < TOL[dtype], (r, err(got[r], want, dtype))
        if alone is not None:   # the same arithmetic without the batch: closer than the bf16 spread
            ref = run_schedule(alone, {r: toks}, [[(r, len(toks))]])[r]
            assert err(got[r], ref, dtype) < 0.1, (r, err(got[r], ref, dtype))


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("block_size", [16, 64])
def test_sink_states_and_block_edges(tmp_path, device, block_size):
    """Sharp attention, slow decays, cuts and decoding at and around the blocks', the chunks' and the query tiles' edges
    (float32); a dropped sink, a dropped gate and a state that starts a portion from zero would show."""
    say("edges", device, block_size)
    cfg = cfg_tiled()
    path, cj, W = checkpoint(cfg, tmp_path, seed=5, sharpen=_sharp)
    toks = tokens(140, cfg.vocab_size, 7)
    want = oracle_logits(cj, W, toks)
    W2 = dict(W)
    W2["l1.mix.sink"] = W["l1.mix.sink"] - 30.0
    assert err(oracle_logits(cj, W2, toks), want) > 50 * TOL["float32"]
    W2 = dict(W)
    W2["l4.mix.g"] = W["l4.mix.g"] * 0
    assert err(oracle_logits(cj, W2, toks), want) > 50 * TOL["float32"]
    assert err(oracle_logits(cj, W, toks[64:]), want[64:]) > 50 * TOL["float32"]     # (everything before token 64 forgotten)
    eng = engine(path, device, "float32", block_size=block_size, blocks=12)
    for cuts in ([32, 1, 1, 106], [31, 33, 76], [64, 64, 12], [63, 1, 1, 1, 74], [65, 2, 73], [15, 1, 1, 1, 46, 32, 32, 12],
                 [2] * 70, [127, 1, 1, 11]):
        assert sum(cuts) == len(toks)
        got = run_schedule(eng, {"a": toks}, [[("a", c)] for c in cuts])["a"]
        assert err(got, want) < TOL["float32"], (cuts, err(got, want))


@pytest.mark.gpu
def test_chunked_and_tiled_kernels_bf16(tmp_path):
    """bfloat16 on the GPU with the shapes the MFMA kernels take: prompts that continue cached context and carried states,
    cut inside chunks, tiles and blocks, against the oracle and against the same engine run whole."""
    cfg = cfg_tiled()
    path, cj, W = checkpoint(cfg, tmp_path, seed=6)
    toks = tokens(200, cfg.vocab_size, 17)
    want = oracle_logits(cj, W, toks)
    eng = engine(path, "cuda", "bfloat16", block_size=64, blocks=8)
    whole = run_schedule(eng, {"a": toks}, [[("a", 200)]])["a"]
    assert err(whole, want) < 0.1, err(whole, want)
    for cuts in ([70, 130], [33, 31, 1, 135], [40, 1, 1, 1, 157], [17] * 11 + [13], [3, 2, 67, 128], [32] * 6 + [8]):
        got = run_schedule(eng, {"a": toks}, [[("a", c)] for c in cuts])["a"]
        assert err(got, want) < 0.1, (cuts, err(got, want))
        assert err(got, whole) < 0.06, (cuts, err(got, whole))


@pytest.mark.parametrize("device", DEVICES)
def test_long_decode_and_far_tokens(tmp_path, device):
    """200 tokens decoded one by one after a short prompt, two sequences of different lengths in the batch; attention and
    the states reach back to the first tokens (the oracle with the first token changed differs at the end)."""
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


@pytest.mark.parametrize("device", DEVICES)
def test_greedy_generation_through_the_scheduler(tmp_path, device):
    """engine.add_request / step(): five requests, three slots, greedy; each output token is the oracle's argmax (tokens
    whose top two logits are closer than the tolerance are skipped)."""
    say("generate", device)
    cfg = cfg_mixed()
    path, cj, W = checkpoint(cfg, tmp_path, seed=11)
    eng = engine(path, device, "float32", blocks=12, seqs=3)
    prompts = [tokens(n, cfg.vocab_size, 30 + i) for i, n in enumerate((5, 19, 2, 33, 11))]
    outs = {}
    for i, p in enumerate(prompts):
        eng.add_request(f"r{i}", p, SamplingParams(max_tokens=12, ignore_eos=True))
    while eng.has_unfinished():
        for o in eng.step():
            if o.finished:
                outs[o.request_id] = list(o.seq.output_ids)
    assert len(eng.blocks.free) == 12 and eng.slots.num_free == 3
    for i, p in enumerate(prompts):
        out = outs[f"r{i}"]
        assert len(out) == 12
        lg = oracle_logits(cj, W, p + out[:-1])[len(p) - 1:]
        for j, t in enumerate(out):
            top = lg[j].topk(2).values
            assert float(lg[j].max() - lg[j][t]) <= 1e-3 * float(lg[j].std()) or float(top[0] - top[1]) < 1e-3, (i, j)


@pytest.mark.gpu
def test_pipelined_decode_takes_the_previous_token_from_the_device(tmp_path):
    """Pipelined decode: a step's input token is the sample the step before left on the device, and the embedding output
    that a loop adds again is that token's; the outputs equal those of the engine that waits for every step."""
    cfg = cfg_mixed()
    path, cj, W = checkpoint(cfg, tmp_path, seed=12)
    prompts = [tokens(n, cfg.vocab_size, 40 + i) for i, n in enumerate((7, 21, 3))]
    outs = {}
    for pipe in (False, True):
        eng = engine(path, "cuda", "float32", blocks=12, seqs=3, pipeline=pipe)
        for i, p in enumerate(prompts):
            eng.add_request(f"r{i}", p, SamplingParams(max_tokens=20, ignore_eos=True))
        res = {}
        while eng.has_unfinished():
            for o in eng.step():
                if o.finished:
                    res[o.request_id] = list(o.seq.output_ids)
        outs[pipe] = res
    assert outs[True] == outs[False] and all(len(v) == 20 for v in outs[True].values())


def test_preempted_requests_start_over_from_zero_states(tmp_path):
    """A pool too small for the decoded tails: a sequence is preempted, its pages and slot are taken by another, and its
    recomputation gives the same tokens as in a pool with room."""
    cfg = cfg_mixed()
    path, cj, W = checkpoint(cfg, tmp_path, seed=13)
    prompts = [tokens(n, cfg.vocab_size, 50 + i) for i, n in enumerate((14, 17, 12))]
    outs = {}
    for blocks in (5, 24):
        eng = engine(path, "cpu", "float32", blocks=blocks, seqs=3)
        for i, p in enumerate(prompts):
            eng.add_request(f"r{i}", p, SamplingParams(max_tokens=30, ignore_eos=True))
        res = {}
        while eng.has_unfinished():
            for o in eng.step():
                if o.finished:
                    res[o.request_id] = list(o.seq.output_ids)
        outs[blocks] = res
        assert len(eng.blocks.free) == blocks and eng.slots.num_free == 3
    assert outs[5] == outs[24] and all(len(v) == 30 for v in outs[5].values())


def test_config_reader_rejects_unknown_keys_and_roundtrips(tmp_path):
    from symmetry_amd.models.weights import safetensors_shapes

    cfg = cfg_mixed()
    path, cj, _ = checkpoint(cfg, tmp_path)
    shapes = safetensors_shapes(path)
    back = C.from_config_json(cj, "t-mixed", shapes)
    assert back == dataclasses.replace(cfg)
    assert back.state_bytes_per_seq() == cfg.state_bytes_per_seq() > 0
    assert C.from_config_json(C.beletar_to_config(cfg_noloop()), "x", {"l2.mix.a1": (1, 28), "l2.mix.g1": (1, 28)}).loop is None

    def bad(change):
        c = copy.deepcopy(cj)
        change(c)
        with pytest.raises(ValueError):
            C.from_config_json(c, "x", shapes)

    bad(lambda c: c["layers"][1]["mixer"].update(chunk=8))
    bad(lambda c: c["layers"][0]["mixer"]["rot"]["scaling"].update(extra=1))
    bad(lambda c: c["layers"][1]["mixer"].update(kv_heads=3))
    bad(lambda c: c["loop"].update(stop=99))
    bad(lambda c: c.update(window=5))
    bad(lambda c: c["layers"][0].update(type="attention"))
    with pytest.raises(ValueError):
        C.from_config_json(cj, "x")              # the ranks are nowhere
    assert C.resolve("tiny-beletar").family == "beletar"


def test_registered_model_by_name_and_checkpoint_tensors(tmp_path):
    """The registry name runs with random weights as every other modelName does (the command line's path), and equals the
    oracle; a checkpoint may carry the second norm of a layer without feed-forward, and no other extra tensor."""
    from safetensors.torch import load_file, save_file

    from symmetry_amd.models.weights import random_weights

    c = C.resolve("tiny-beletar")
    eng = LLMEngine(EngineConfig(model="tiny-beletar", weights="random", dtype="float32", device="cpu", max_num_seqs=2,
                                 block_size=16, num_kv_blocks=9, max_model_len=128, use_graphs=False,
                                 enable_prefix_caching=False, pipeline=False, seed=3))
    W = {k: v.to(torch.bfloat16) for k, v in random_weights(c, seed=3).tensors.items()}
    toks = tokens(50, c.vocab_size, 2)
    got = run_schedule(eng, {"a": toks}, [[("a", 31)], [("a", 19)]])["a"]
    assert err(got, oracle_logits(C.beletar_to_config(c), W, toks)) < TOL["float32"]
    cfg = cfg_mixed()
    path, cj, W = checkpoint(cfg, tmp_path, seed=4)
    f = os.path.join(path, "model.safetensors")
    t = load_file(f)
    t["l3.norm2"], t["l3.norm2.b"] = torch.ones(cfg.hidden_size), torch.zeros(cfg.hidden_size)
    save_file(t, f)
    toks = tokens(20, cfg.vocab_size, 5)
    got = run_schedule(engine(path, "cpu", "float32"), {"a": toks}, [[("a", 20)]])["a"]
    assert err(got, oracle_logits(cj, W, toks)) < TOL["float32"]
    t["l3.mix.q.b"] = torch.ones(4)
    save_file(t, f)
    with pytest.raises(ValueError):
        engine(path, "cpu", "float32")
    del t["l3.mix.q.b"], t["l1.mix.A_log"]
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


def _two_runs(na, nb, first_a, first_b, slot_a=2, slot_b=0):
    """Step metadata of sequence a's rows beside sequence b's: prev_row, save_slot, row_seq, cu_q, runs, 64-row tiles."""
    prev, save, rs, cu, tiles = [], [], [], [0], []
    r0 = 0
    for cnt, first, slot in ((na, first_a, slot_a), (nb, first_b, slot_b)):
        if not cnt:
            continue
        prev += [-1 if first else -(slot + 2)] + list(range(r0, r0 + cnt - 1))
        save += [-1] * (cnt - 1) + [slot]
        rs += [len(cu) - 1] * cnt
        tiles += [[len(cu) - 1, o] for o in range(0, cnt, 64)]
        r0 += cnt
        cu.append(r0)
    i32 = torch.int32
    tiles.append([0, 1 << 20])      # a padding tile
    return (torch.tensor(prev, dtype=i32), torch.tensor(save, dtype=i32), torch.tensor(rs, dtype=i32),
            torch.tensor(cu, dtype=i32), len(cu) - 1, torch.tensor(tiles, dtype=i32))


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("d", [24, 301, 2048, 2500, 8200])
def test_residual_sum_with_the_next_layer_norm(device, d):
    """x = base + a + b and the layer norm with weight and bias from the same pass; rows far from mean zero; the sum alone;
    the gathered norm in front of the head."""
    say("op residual_layer_norm", device, d)
    torch.manual_seed(d)
    for T in (3, 300):
        base, a, b = torch.randn(T, d) + 5.0, torch.randn(T, d), torch.randn(T, d).to(torch.bfloat16)
        w, bias = torch.rand(d) + 0.5, torch.randn(d)
        x = torch.full((T, d), 1e4)
        x, base_d, a_d, b_d, wd, bd = _dev(device, x, base, a, b, w, bias)
        h = torch.empty(T, d, device=device)
        ops.residual_layer_norm(x, a_d, b_d, wd, bd, 1e-5, None, h, base=base_d)
        want = base.double() + a.double() + b.double()
        assert float((x.cpu().double() - want).abs().max()) < 1e-5
        assert float((h.cpu().double() - O.layer_norm(want, w.double(), bias.double(), 1e-5)).abs().max()) < 2e-5
        ops.residual_layer_norm(x, a_d)                                    # the last sublayer's sum
        want = want + a.double()
        assert float((x.cpu().double() - want).abs().max()) < 1e-5
        hb = torch.empty(T, d, device=device, dtype=torch.bfloat16)
        ops.residual_layer_norm(x, w=wd, bias=bd, eps=1e-5, out=hb)        # the norm alone
        full = O.layer_norm(want, w.double(), bias.double(), 1e-5)
        assert float((hb.cpu().double() - full).abs().max()) < 2e-2 * float(full.abs().max())
        rows = torch.tensor([T - 1, 0], device=device)
        out = torch.empty(2, d, device=device)
        ops.residual_layer_norm(x, w=wd, bias=bd, eps=1e-5, rows=rows, out=out)
        assert float((out.cpu().double() - full[rows.cpu()]).abs().max()) < 2e-5


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("taps", [1, 2, 3, 4, 7, 16])
@pytest.mark.parametrize("shape", [(2, 5, 3, 7), (1, 8, 2, 12), (2, 64, 2, 300)])
def test_convolved_projections_with_carried_taps(device, taps, shape):
    """q | k | v through the short convolution and silu over runs that continue a sequence through its state slot, queries
    and keys brought to unit length per head: whatever the cut, the whole-sequence result."""
    G, N, H, P = shape
    say("op conv_silu_qkv", device, taps, shape)
    torch.manual_seed(taps)
    n, nb = 41, 9
    C_ = 2 * G * N + H * P
    za, zb, w = torch.randn(n, C_ + 8), torch.randn(nb, C_ + 8), torch.randn(C_, taps) * 0.7
    za[4, :G * N] *= 1e-3        # a short query: the length's epsilon shows

    def whole(z):
        y = O.silu(O.short_conv(z[:, :C_].double(), w.double()))
        q, k = O.unit(y[:, :G * N].view(-1, G, N)) * 0.3, O.unit(y[:, G * N:2 * G * N].view(-1, G, N))
        return torch.cat([q.flatten(1), k.flatten(1), y[:, 2 * G * N:]], 1)

    want_a, want_b = whole(za), whole(zb)
    state = torch.full((3, taps - 1, C_), 1e4)
    state, wd = _dev(device, state, w)
    got_a, got_b = [], []
    at_a = at_b = 0
    for na, nb_, decode in ((3, 2, False), (1, 1, True), (1, 1, True), (taps, 0, False), (1, 1, True), (19 - taps, 3, False),
                            (1, 1, True), (15, 0, False)):
        prev, save, rs, cu, runs, _ = _two_runs(na, nb_, at_a == 0, at_b == 0)
        T = na + nb_
        z = torch.cat([za[at_a:at_a + na], zb[at_b:at_b + nb_]])
        q, k, v = torch.empty(T, G, N), torch.empty(T, G, N), torch.empty(T, H, P)
        z, q, k, v, prev, save, rs, cu = _dev(device, z, q, k, v, prev, save, rs, cu)
        zin = z[:, :C_]
        if decode:      # (with a small projection of another input in the same launch)
            x, gw = torch.randn(T, 70), torch.randn(5, 66)
            xd, gwd, go = _dev(device, x, gw, torch.empty(T, 5))
            ops.conv_silu_qkv(zin, wd, state, None, None, prev, T, G, N, H, P, 0.3, 1e-6, q, k, v, save_slot=save,
                              gates=(xd[:, :66], gwd, go))
            assert float((go.cpu().double() - x[:, :66].double() @ gw.double().T).abs().max()) < 1e-4
        else:
            ops.conv_silu_qkv(zin, wd, state, cu, rs, prev, runs, G, N, H, P, 0.3, 1e-6, q, k, v)
            if taps > 1:
                ops.conv_state_update(zin, state, cu, prev, save, runs)
        out = torch.cat([q.flatten(1), k.flatten(1), v.flatten(1)], 1).cpu()
        got_a.append(out[:na])
        got_b.append(out[na:])
        at_a, at_b = at_a + na, at_b + nb_
    assert float((torch.cat(got_a).double() - want_a[:at_a]).abs().max()) < 1e-4
    assert float((torch.cat(got_b).double() - want_b[:at_b]).abs().max()) < 1e-4
    if taps > 1:
        assert float(state[1].min()) == 1e4        # the unused slot was never written


@pytest.mark.parametrize("device", DEVICES)
def test_convolved_projections_long_prompt_bf16(device):
    """A prompt step of hundreds of rows in bfloat16: two runs in one step, the second continuing its sequence from the
    slot, run borders inside a wave's rows."""
    say("op conv_silu_qkv long", device)
    torch.manual_seed(11)
    G, N, H, P, taps = 2, 32, 4, 48, 4
    C_ = 2 * G * N + H * P
    na, nb = 403, 122
    bf = torch.bfloat16
    za, zb, w = torch.randn(na, C_).to(bf), torch.randn(nb + 3, C_).to(bf), (torch.randn(C_, taps) * 0.7).to(bf)
    y = O.silu(torch.cat([O.short_conv(za.double(), w.double()), O.short_conv(zb.double(), w.double())[3:]]))
    state = torch.full((3, taps - 1, C_), 1e4, dtype=bf)
    state[0] = zb[:3]
    prev, save, rs, cu, runs, _ = _two_runs(na, nb, True, False)
    T = na + nb
    z, q, k, v = torch.cat([za, zb[3:]]), torch.empty(T, G, N), torch.empty(T, G, N), torch.empty(T, H, P, dtype=bf)
    z, wd, state, q, k, v, prev, save, rs, cu = _dev(device, z, w, state, q, k, v, prev, save, rs, cu)
    ops.conv_silu_qkv(z, wd, state, cu, rs, prev, runs, G, N, H, P, N ** -0.5, 1e-6, q, k, v)
    ops.conv_state_update(z, state, cu, prev, save, runs)
    assert float((q.cpu().double() - O.unit(y[:, :G * N].view(T, G, N)) * N ** -0.5).abs().max()) < 1e-5
    assert float((k.cpu().double() - O.unit(y[:, G * N:2 * G * N].view(T, G, N))).abs().max()) < 1e-5
    assert float((v.cpu().double() - y[:, 2 * G * N:].view(T, H, P)).abs().max()) < 3e-2
    assert torch.equal(state[0].cpu(), zb[-3:]) and torch.equal(state[2].cpu(), za[-3:])


def _delta_case(channel, H, G, N, P, n, seed, strong=False):
    torch.manual_seed(seed)
    q, k = O.unit(torch.randn(n, G, N)) * N ** -0.5, O.unit(torch.randn(n, G, N) + 0.3)
    v, bz = torch.randn(n, H, P), torch.randn(n, H)
    # the first token writes a key that no other one touches, and the last token asks for it
    k[:, :, 0] = 0.0
    k[0] = torch.eye(N)[0]
    k, q[-1] = O.unit(k), torch.eye(N)[0]
    cols = H * N if channel else H
    dz, dtb = torch.randn(n, cols) * (3.0 if strong else 1.0), torch.randn(cols) - (0.0 if strong else 6.0)
    A = torch.randn(H) * (1.5 if strong else 0.3)
    if strong:
        A[0] = 1.5
        dz[5], dz[40], dz[7] = 40.0, 40.0, -40.0
    lg = -torch.exp(A.double())[None, :, None] * O.softplus((dz + dtb).double().view(n, H, -1)).expand(n, H, N)
    want, S = O.delta_rule(q.double(), k.double(), v.double(), lg, torch.sigmoid(bz.double()))
    return q, k, v, dz, dtb, A, bz, lg, want, S


FORMS = [("cpu", 1), pytest.param("cuda", 1, marks=pytest.mark.gpu), pytest.param("cuda", 0, marks=pytest.mark.gpu)]


@pytest.mark.parametrize("device,impl", FORMS)
@pytest.mark.parametrize("channel", [False, True])
@pytest.mark.parametrize("shape", [(3, 1, 9, 5), (2, 2, 16, 33), (4, 2, 40, 20), (2, 1, 64, 70), (1, 1, 130, 16), (1, 1, 256, 8)])
def test_delta_rule_handed_over_through_slots(device, impl, channel, shape):
    """The recurrence over runs cut anywhere (prompt runs beside single rows), states handed over through slots with garbage
    in the unused one, decays slow enough that the first token still counts at the end; token by token and chunked."""
    H, G, N, P = shape
    say("op delta_rule", device, impl, channel, shape)
    na_all, nb_all = 117, 45
    qa, ka, va, dza, dtb, A, bza, lga, want_a, Sa = _delta_case(channel, H, G, N, P, na_all, 1)
    qb, kb, vb, dzb, _, _, bzb, _, _, _ = _delta_case(channel, H, G, N, P, nb_all, 2)
    lgb = -torch.exp(A.double())[None, :, None] * O.softplus((dzb + dtb).double().view(nb_all, H, -1)).expand(nb_all, H, N)
    want_b, Sb = O.delta_rule(qb.double(), kb.double(), vb.double(), lgb, torch.sigmoid(bzb.double()))
    va2 = va.clone()
    va2[0] += 3.0
    far, _ = O.delta_rule(qa.double(), ka.double(), va2.double(), lga, torch.sigmoid(bza.double()))
    assert float((far[-1] - want_a[-1]).abs().max()) > 0.05       # (the tolerance below is 4e-6)
    state = torch.full((3, H, N, P), 1e4)
    state, dtb_d, A_d = _dev(device, state, dtb, A)
    got_a, got_b = [], []
    at_a = at_b = 0
    for na, nb, decode in ((7, 3, False), (1, 1, True), (1, 1, True), (32, 0, False), (2, 33, False), (65, 2, False), (1, 5, False),
                           (8, 0, False)):
        prev, save, rs, cu, runs, tiles = _two_runs(na, nb, at_a == 0, at_b == 0)
        cat = [torch.cat([x[at_a:at_a + na], y[at_b:at_b + nb]]) for x, y in ((qa, qb), (ka, kb), (va, vb), (dza, dzb), (bza, bzb))]
        T = na + nb
        y = torch.full((T, H, P), 1e4)
        ws = torch.full((T, H, ops.delta_ws_cols(channel, N)), float("nan"))
        q, k, v, dz, bz, y, ws, prev, save, cu, tiles = _dev(device, *cat, y, ws, prev, save, cu, tiles)
        chunked = impl == 0 and not decode
        used = ops.delta_rule(channel, q, k, v, dz, dtb_d, A_d, bz, state, None if decode else cu, prev, save,
                              T if decode else runs, y, tiles if chunked else None, ws if chunked else None)
        assert used == (0 if chunked else 1)
        got_a.append(y[:na].cpu())
        got_b.append(y[na:].cpu())
        at_a, at_b = at_a + na, at_b + nb
    assert (at_a, at_b) == (na_all, nb_all)
    assert float((torch.cat(got_a).double() - want_a).abs().max()) < 4e-6
    assert float((torch.cat(got_b).double() - want_b).abs().max()) < 4e-6
    assert float((state[2].cpu().double() - Sa).abs().max()) < 2e-5 and float((state[0].cpu().double() - Sb).abs().max()) < 2e-5
    assert float(state[1].min()) == 1e4            # the unused slot was never written


@pytest.mark.parametrize("device,impl", FORMS)
@pytest.mark.parametrize("channel", [False, True])
def test_delta_rule_strong_decays_and_one_key_again(device, impl, channel):
    """Decays from none to complete within a chunk (nothing overflows), and a key written twice: with beta near one the
    second value replaces the first, whether the two writes share a chunk or not."""
    say("op delta_rule strong", device, impl, channel)
    H, G, N, P, n = 2, 1, 32, 24, 100
    q, k, v, dz, dtb, A, bz, lg, want, S = _delta_case(channel, H, G, N, P, n, 3, strong=True)
    assert float(lg.min()) < -100.0 and float(lg.max()) > -1e-3

    def run(q, k, v, dz, dtb, A, bz):
        prev, save, rs, cu, runs, tiles = _two_runs(n, 0, True, True)
        state, y = torch.zeros(3, H, N, P), torch.empty(n, H, P)
        ws = torch.full((n, H, ops.delta_ws_cols(channel, N)), float("nan"))
        q, k, v, dz, dtb, A, bz, state, y, ws, prev, save, cu, tiles = _dev(device, q, k, v, dz, dtb, A, bz, state, y, ws, prev,
                                                                            save, cu, tiles)
        ops.delta_rule(channel, q, k, v, dz, dtb, A, bz, state, cu, prev, save, runs, y, tiles if impl == 0 else None,
                       ws if impl == 0 else None)
        return y.cpu()

    got = run(q, k, v, dz, dtb, A, bz)
    assert float((got.double() - want).abs().max()) < 2e-6 * max(1.0, float(want.abs().max()))
    for first, second, ask in ((3, 9, 20), (3, 40, 41), (31, 32, 99), (10, 63, 64)):
        k2 = torch.zeros(n, G, N)
        k2[:, :, 0] = 1.0                        # every other token writes key 0 with a zero step
        k2[first], k2[second] = torch.eye(N)[5], torch.eye(N)[5]
        q2 = torch.zeros(n, G, N)
        q2[ask, :, 5] = 1.0
        bz2 = torch.full((n, H), -40.0)
        bz2[first], bz2[second] = 40.0, 40.0
        none = torch.full_like(dz, -40.0)        # no decay
        y = run(q2, k2, v, none, torch.zeros_like(dtb), torch.zeros(H), bz2)
        assert float((y[ask] - v[second]).abs().max()) < 1e-5, (first, second, ask)


@pytest.mark.parametrize("device", DEVICES)
def test_head_norm_with_either_gate(device):
    say("op gated_group_norm", device)
    torch.manual_seed(5)
    T, H, P = 7, 3, 22
    y, gate, w = torch.randn(T, H * P), torch.randn(T, H * P + 4), torch.rand(P) + 0.5
    for sigmoid in (False, True):
        g = gate[:, :H * P].double()
        want = O.rms_norm(y.double().view(T, H, P), w.double(), 1e-5).reshape(T, -1) * (torch.sigmoid(g) if sigmoid else O.silu(g))
        yd, gd, wd, out = _dev(device, y, gate, w, torch.empty(T, H * P))
        ops.gated_group_norm(yd, gd[:, :H * P], wd, 1e-5, P, False, out, sigmoid=sigmoid)
        assert float((out.cpu().double() - want).abs().max()) < 1e-5


@pytest.mark.parametrize("scaling", [None, (3.0, 40.0, 4.0, 0.5), (8.0, 5000.0, 32.0, 1.0), (2.0, 7.0, 1.2, 1.0)])
def test_blended_rotary_table(scaling):
    """The table's angles and magnitude against the oracle's (ramps inside, before and past the pairs, a ramp of width
    zero)."""
    rot = {"base": 300.0, "dims": 16}
    if scaling:
        rot["scaling"] = dict(zip(("factor", "original", "fast", "slow"), scaling))
    pos = torch.arange(50)
    a, mag = O.rotation_angles(pos, rot)
    t = ops.rope_scaled_table(50, 16, 300.0, *(scaling or ()))
    assert float((t[..., 0].double() - torch.cos(a) * mag).abs().max()) < 2e-5
    assert float((t[..., 1].double() - torch.sin(a) * mag).abs().max()) < 2e-5


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("shape", [(4, 48, 16, 24), (20, 24, 8, 6), (3, 21, 6, 10)])
def test_latent_attention_with_sink_and_head_gate(device, dtype, shape):
    """Cache rows written through a shuffled block table; one query looks hard at one key (the first, at block borders, far
    back, itself); per-head sink and gate; prompt rows, single rows with and without split-KV partitions."""
    if device == "cpu" and dtype == torch.bfloat16:
        pytest.skip("the reference op is the float32 one")
    H, r, rot, dv = shape
    say("op latent_attn sink gate", device, dtype, shape)
    torch.manual_seed(4)
    n, BS, scale = 150, 16, 0.4
    Dk = r + rot
    NB, bt, pos, slots = _paged(n, BS, 9)
    zc, wkv = torch.randn(n, Dk + 8), torch.rand(r) + 0.5
    table = ops.rope_scaled_table(256, rot, 100.0, 4.0, 64.0, 8.0, 1.0)
    sink = torch.linspace(-1.0, 2.5, H)
    gate = torch.randn(n, H + 8)
    tol = 2e-5 if dtype == torch.float32 else 4e-2
    cache = torch.zeros(NB, BS, Dk, dtype=dtype)
    zc, wkv, table, cache, slots_d, posd = _dev(device, zc.to(dtype), wkv.to(dtype), table, cache, slots, pos)
    ops.latent_prep(zc[:, :Dk], 0, r, rot, None, wkv, 1e-6, posd, slots_d, table, None, cache)
    rows = cache.cpu().view(-1, Dk)[slots.long()].double()
    rotd = {"base": 100.0, "dims": rot, "scaling": {"factor": 4.0, "original": 64.0, "fast": 8.0, "slow": 1.0}}
    zf = zc.cpu().double()
    want_rows = torch.cat([O.rms_norm(zf[:, :r], wkv.cpu().double(), 1e-6), O.rotate_pairs(zf[:, r:Dk], pos, rotd)], 1)
    assert float((rows - want_rows).abs().max()) < (1e-5 if dtype == torch.float32 else 3e-2)
    i = torch.arange(n)
    for target in (0, 1, 15, 16, 127, 128, 149):
        q = torch.randn(n, H, Dk) * 0.1
        q[149] = rows[target].float() * (9.0 / scale) / float(rows[target].pow(2).sum())
        q = q.to(dtype)
        s = torch.einsum("thd,sd->hts", q.double(), rows) * scale
        s = s.masked_fill(i[:, None] < i[None, :], float("-inf"))
        g = torch.sigmoid(gate[:, :H].to(dtype).double())
        want = torch.einsum("hts,sr->thr", O.sink_softmax(s, sink.double()), rows[:, :r]) * g[:, :, None]
        cu, rs = torch.tensor([0, n], dtype=torch.int32), torch.zeros(n, dtype=torch.int32)
        tiles = torch.tensor([[0, o] for o in range(0, n, 64)], dtype=torch.int32)
        out = torch.empty(n, H, r, dtype=dtype)
        qd, btd, rsd, sd, gd, out, cud, tilesd = _dev(device, q, bt, rs, sink, gate.to(dtype), out, cu, tiles)
        gv = gd[:, :H]
        impl = ops.latent_attn(qd, cache, btd, rsd, posd, scale, r, out, None, None, tilesd, cud, sink=sd, gate=gv)
        mfma = device != "cpu" and dtype == torch.bfloat16 and Dk % 32 == 0 and r % 16 == 0
        assert impl == (0 if mfma else 1)
        assert float((out.cpu().double() - want).abs().max()) < tol, target
        for parts in (1, 4):
            one = torch.empty(1, H, r, dtype=dtype, device=device)
            po = pm = None
            if parts > 1 and device != "cpu":
                po = torch.empty(1, H, parts, r, device=device)
                pm = torch.empty(1, H, parts, 2, device=device)
            ops.latent_attn(qd[149:].clone(), cache, btd, rsd[:1], posd[149:], scale, r, one, po, pm, sink=sd, gate=gv[149:])
            assert float((one.cpu().double() - want[149:]).abs().max()) < tol, (target, parts)
    plain = torch.empty(1, H, r, dtype=dtype, device=device)
    ops.latent_attn(qd[5:6].clone(), cache, btd, rsd[:1], posd[5:6], scale, r, plain, gate=gv[5:6])     # (a row with few keys)
    assert float((plain.cpu().double() - want[5:6]).abs().max()) > 4 * tol
    ops.latent_attn(qd[5:6].clone(), cache, btd, rsd[:1], posd[5:6], scale, r, plain, sink=sd)
    assert float((plain.cpu().double() - want[5:6]).abs().max()) > 4 * tol
    huge = torch.full_like(sd, 200.0)       # a sink that takes everything: no overflow, an output of zero
    ops.latent_attn(qd[5:6].clone(), cache, btd, rsd[:1], posd[5:6], scale, r, plain, sink=huge)
    assert float(plain.abs().max()) < 1e-6


@pytest.mark.parametrize("device", DEVICES)
def test_silu_gated_product_and_unrounded_linear(device):
    say("op silu_mul linear_f32", device)
    torch.manual_seed(6)
    for F, dt, tol in ((24, torch.float32, 1e-5), (24, torch.bfloat16, 3e-2), (21, torch.bfloat16, 3e-2)):
        gu = torch.randn(5, 2 * F).to(dt)
        gud, out = _dev(device, gu, torch.empty(5, F, dtype=dt))
        ops.silu_mul(gud[:, :F], gud[:, F:], out)
        want = O.silu(gu[:, :F].double()) * gu[:, F:].double()
        assert float((out.cpu().double() - want).abs().max()) < tol
    for dt in (torch.float32, torch.bfloat16):
        x, w = torch.randn(9, 40).to(dt), torch.randn(6, 40).to(dt)
        xd, wd, out = _dev(device, x, w, torch.empty(9, 6))
        ops.linear_f32(xd, wd, out)
        assert float((out.cpu().double() - x.double() @ w.double().T).abs().max()) < 1e-4
