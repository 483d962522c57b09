"""Kosusun through the engine's own logic on the CPU (the kernel library replaced by the plain-torch
stand-in of tests/cpu_ops.py): configuration and weights, two groups of pages (a window's and its
pooled blocks') and state slots, all ways of cutting the work, pages and slots that change hands,
and greedy generation through the scheduler, against the plain implementation; and the plain
implementation's own facts by hand."""
import json
import math

import numpy as np
import pytest
import torch

import plain_kosusun
from cpu_ops import CpuOps
from helpers import collect, max_error, random_prompt, trace_mixed, trace_portions, trace_prefill_then_decode, trace_whole
from kosusun_helpers import (SMALL, _config, _layer, _mlstm, _parallel, _retention, _rot, _window, make_weights, plain_greedy, plain_logits,
                             write_folder)
from tiny_llm_infer_amd.cache.manager import PAGE, CacheFull, CacheManager, CacheNeed, CacheRecord
from tiny_llm_infer_amd.config import ConfigError, KosusunConfig
from tiny_llm_infer_amd.engine.llm_engine import LLMEngine
from tiny_llm_infer_amd.engine.loading import load_model
from tiny_llm_infer_amd.engine.replay import Replayer
from tiny_llm_infer_amd.engine.runner import ModelRunner
from tiny_llm_infer_amd.registry import architecture_of
from tiny_llm_infer_amd.sampling.params import SamplingParams
from tiny_llm_infer_amd.weights.loader import WeightError

F64 = torch.float64


@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    root = tmp_path_factory.mktemp("kosusun")
    return {name: write_folder(str(root / name), cfg, make_weights(cfg, seed)) for name, (cfg, _, seed) in SMALL.items()}


def _runner(folder, page, max_tokens, max_requests=4):
    model, _ = load_model(folder, "float32", "cpu", max_model_len=1024, ops=CpuOps())
    return ModelRunner(model, model.env, page_size=page, num_pages=max_tokens // page,
                       max_requests=max_requests, max_batch_tokens=512)


def _replay(runner, steps):
    rp = Replayer(runner)
    return {st["step"]: rp.run_step(st) for st in steps}


def _requests(name, lengths, seed):
    vocab = SMALL[name][0]["vocab"]
    return {f"r{i}": random_prompt(vocab, n, seed + i) for i, n in enumerate(lengths)}


# ------------------------------------------------------------ configuration ---
def test_config_round_trip_and_registry():
    from tiny_llm_infer_amd.models.kosusun import kosusun_spec
    for name, (cfg, _, _) in SMALL.items():
        typed = KosusunConfig.from_dict(cfg)
        assert typed.to_dict() == cfg
        assert architecture_of(cfg).name == "Kosusun"
        spec = kosusun_spec(typed)
        assert [c.block for c in spec.schedule] == list(range(len(cfg["layers"])))
        kept = [c.cache for c, layer in zip(spec.schedule, cfg["layers"]) if layer["type"] == "parallel"]
        assert kept == list(range(len(kept)))
        assert {b.arrangement for b in spec.blocks} == {"parallel_one_norm"}


@pytest.mark.parametrize("change, message", [
    (lambda c: c.pop("width"), "width"),
    (lambda c: c["layers"][0].update(type="conv"), "layer type"),
    (lambda c: c["layers"][0]["mixer"]["left"].update(kv_heads=3), "multiple"),
    (lambda c: c["layers"][0]["mixer"]["left"]["mask"].update(pool=0), "pool"),
    (lambda c: c["layers"][0]["mixer"]["left"]["mask"].pop("size"), "size"),
    (lambda c: c["layers"][0]["mixer"]["left"]["rot"].update(dims=7), "rot.dims"),
    (lambda c: c["layers"][0]["mixer"]["left"]["rot"]["scaling"].update(factor=0.0), "factor"),
    (lambda c: c["layers"][0]["mixer"]["left"].pop("scale"), "scale"),
    (lambda c: c["layers"][0]["mixer"]["right"]["rot"].update(dims=14), "rot.dims"),
    (lambda c: c["layers"][0]["mixer"]["right"].update(decay=[0.5]), "one a head"),
    (lambda c: c["layers"][0]["mixer"].pop("left_scale"), "left_scale"),
    (lambda c: c["layers"][1]["mixer"].update(gate_cap=0.0), "gate_cap"),
    (lambda c: c["layers"][1]["mlp"].update(kind="moe"), "feed-forward kind"),
    (lambda c: c["norm"].update(eps=0.0), "eps"),
])
def test_config_errors(change, message):
    cfg = json.loads(json.dumps(SMALL["A"][0]))
    change(cfg)
    with pytest.raises(ConfigError, match=message):
        KosusunConfig.from_dict(cfg)


def test_a_checkpoint_that_does_not_fit_is_refused(tmp_path):
    cfg, _, seed = SMALL["A"]
    w = make_weights(cfg, seed)
    del w["l0.mix.left.sink"]
    w["l1.mix.f"] = w["l1.mix.f"][:-1]
    w["l0.norm2"] = w["l0.norm1"].clone()
    folder = write_folder(str(tmp_path / "bad"), cfg, w)
    with pytest.raises(WeightError) as err:
        load_model(folder, "float32", "cpu", ops=CpuOps())
    assert err.value.missing == ["l0.mix.left.sink"] and err.value.unexpected == ["l0.norm2"]
    assert [n for n, _, _ in err.value.wrong_shape] == ["l1.mix.f"]


# ---------------------------------------------------- pages with one slot for several positions ---
def test_groups_of_a_window_and_of_its_blocks(folders):
    runner = _runner(folders["A"], 16, 256)
    window, blocks = runner.cache.groups
    assert (window.need.window, window.need.stride) == (20, 1) and (blocks.need.window, blocks.need.stride) == (None, 4)
    assert window.need.records == blocks.need.records
    # 16 pages of 16 tokens: a quarter as many for the blocks, and one that each of four requests has begun
    assert runner.cache.pages_per_group() == [16, 4 + 4]
    states = [s for s in runner.states if s is not None]
    assert [set(s) for s in states] == [{"right"}, {"S", "m"}, {"S", "m"}]
    assert tuple(states[0]["right"].shape) == (5, 3, 20, 12) and tuple(states[1]["S"].shape) == (5, 2, 25, 16)
    # blocks longer than the window: the tokens of a block that is not whole yet are kept
    runner = _runner(folders["B"], 8, 128)
    assert [(g.need.window, g.need.stride) for g in runner.cache.groups] == [(10, 1), (24, 1), (None, 10), (None, 5)]


def test_manager_with_strides():
    record = (CacheRecord("k", (1, PAGE, 4)),)
    m = CacheManager([CacheNeed(record, window=10), CacheNeed(record, stride=3)], page_size=4, num_pages=30, max_requests=2,
                     max_step_tokens=20)
    assert m.pages_per_group() == [min(30, 2 * (3 + 2) + 5), 10 + 2]
    m.admit("a")
    assert m.pages_needed("a", 13) == [4, 2]                         # 13 positions: a page of blocks covers 12
    m.reserve("a", 13)
    m.advance("a", 13)
    m.check()
    assert list(m.get("a").tables[0]) == [-1, 1, 2, 3] and list(m.get("a").tables[1]) == [0, 1]      # 13: reads 4..13
    assert m.pages_needed("a", 24) == [2, 0] and m.pages_needed("a", 25) == [3, 1]
    assert m.most_pages_needed(25, 20) == [7, 3]
    m.admit("b")
    with pytest.raises(CacheFull):
        m.reserve("b", 12 * 11)                                      # 11 pages of blocks, 10 are free
    m.reserve("b", 12 * 10 - 108)
    m.release("a")
    m.release("b")
    m.check()
    assert m.free_pages() == m.pages_per_group()
    with pytest.raises(ValueError, match="slot for every position"):
        CacheManager([CacheNeed(record, stride=3)], 4, 30, 2, prefix_caching=True)
    with pytest.raises(ValueError, match="at least one position"):
        CacheNeed(record, stride=0)


def test_page_sizing_counts_a_share_of_a_page_of_blocks(folders):
    from tiny_llm_infer_amd.engine.sizing import estimate_num_pages, page_bytes, window_bytes
    model, _ = load_model(folders["A"], "float32", "cpu", max_model_len=256, ops=CpuOps())
    page = 16 * 4 * 2 * (16 + 24)                                    # of the tokens, and of the blocks
    assert page_bytes(model, 16, windowed=True) == page and page_bytes(model, 16, windowed=False) == page // 4
    assert window_bytes(model, 16, 64, 3) == (3 * (2 + 2) + 4) * page + 3 * page
    assert estimate_num_pages(model, 16, 64, 3, 256) == 3 * 16


# ------------------------------------------------------------------ all the cuts ---
@pytest.mark.parametrize("name", list(SMALL))
def test_all_cuts_match_plain(folders, name):
    folder = folders[name]
    reqs = _requests(name, [70, 45, 97, 33, 1, 58, 2], seed=5)
    want = plain_logits(folder, reqs)
    max_tokens = 256
    cuts = {
        "whole": trace_whole(reqs),
        "decode": trace_prefill_then_decode(reqs),
        "portions": trace_portions(reqs, seed=3),
        "mixed": trace_mixed(reqs, max_tokens=max_tokens, seed=9),
    }
    for cut, steps in cuts.items():
        runner = _runner(folder, SMALL[name][1], max_tokens)
        got = collect(steps, _replay(runner, steps))
        for rid in reqs:
            err, row, scale = max_error(got[rid], want[rid])
            assert err <= 2e-5 * max(1.0, scale), f"{name}/{cut}/{rid}: error {err} at token {row}"
        runner.cache.check()
        assert not runner.cache.live()
        assert runner.cache.free_pages() == runner.cache.pages_per_group()


def test_token_by_token_equals_whole(folders):
    """Every token decoded alone from position 0 against the whole prompt."""
    for name in ("A", "B"):
        folder = folders[name]
        reqs = _requests(name, [60], seed=21)
        want = plain_logits(folder, reqs)
        steps = trace_prefill_then_decode(reqs, tail=59)
        runner = _runner(folder, SMALL[name][1], 64)
        got = collect(steps, _replay(runner, steps))
        err, row, scale = max_error(got["r0"], want["r0"])
        assert err <= 2e-5 * scale, (name, err, row)


def test_pages_and_slots_that_change_hands_carry_nothing_over(folders):
    """Few pages and one state slot, used by request after request; portions down to two tokens."""
    folder = folders["B"]
    reqs = _requests("B", [37, 29, 41], seed=40)
    want = plain_logits(folder, reqs)
    runner = _runner(folder, 8, 48, max_requests=1)
    for tensors in runner.group_tensors:
        for t in tensors.values():
            t.fill_(3.0)                                             # what other requests left
    for s in runner.states:
        for t in s.values():
            t.fill_(-5.0)
    steps = trace_portions(reqs, seed=1)
    got = collect(steps, _replay(runner, steps))
    for rid in reqs:
        err, row, scale = max_error(got[rid], want[rid])
        assert err <= 2e-5 * scale, (rid, err, row)
    assert runner.cache.pages_taken_total > runner.cache.num_pages


def test_the_window_group_gives_pages_back_and_the_blocks_stay(folders):
    folder = folders["A"]
    reqs = _requests("A", [200], seed=2)
    want = plain_logits(folder, reqs)
    runner = _runner(folder, 16, 208)
    steps = trace_prefill_then_decode(reqs, tail=60)[:-1]
    got = collect(steps, _replay(runner, steps))
    window, blocks = runner.cache.get("r0").tables
    assert sum(p >= 0 for p in window) <= 3 and all(p >= 0 for p in blocks) and len(blocks) == 4      # 199 tokens, 64 a page
    err, row, scale = max_error(got["r0"], want["r0"][:-1])
    assert err <= 2e-5 * scale, (err, row)


def test_unequal_requests_together_equal_each_alone(folders):
    folder = folders["R"]
    reqs = _requests("R", [3, 130, 34, 65], seed=60)
    alone = {}
    for rid, toks in reqs.items():
        runner = _runner(folder, 32, 256)
        alone[rid] = _replay(runner, trace_whole({rid: toks}))[0]
    runner = _runner(folder, 32, 512)
    step = {"step": 0, "entries": [{"id": r, "tokens": t, "want": list(range(len(t)))} for r, t in reqs.items()],
            "end": list(reqs)}
    together = collect([step], _replay(runner, [step]))
    for rid in reqs:
        assert np.abs(together[rid] - alone[rid]).max() <= 1e-5 * np.abs(alone[rid]).max()      # (the stand-in's products round by their shape)


# ------------------------------------------------- generation through the scheduler ---
@pytest.mark.parametrize("name", ["A", "B"])
def test_greedy_generation_matches_plain(folders, name):
    folder = folders[name]
    vocab = SMALL[name][0]["vocab"]
    prompts = [random_prompt(vocab, n, 40 + n) for n in (5, 17, 33)]
    want = [plain_greedy(folder, p, 12) for p in prompts]
    args = dict(dtype="float32", device="cpu", max_model_len=128, page_size=SMALL[name][1], num_kv_blocks=64,
                max_num_seqs=4, max_num_batched_tokens=24, ops=CpuOps())
    eng = LLMEngine.from_folder(folder, **args)
    got = eng.generate(prompts, SamplingParams(max_tokens=12, ignore_eos=True))
    assert [r.token_ids for r in got] == want
    eng.runner.cache.check()
    assert eng.runner.cache.free_pages() == eng.runner.cache.pages_per_group()


def test_a_model_that_keeps_state_only(tmp_path):
    """mLSTM layers alone: no group of pages at all, requests live by their slots."""
    cfg = _config(97, 40, [_layer("mlstm", _mlstm(2, 12, 9, 7.0), 33), _layer("mlstm", _mlstm(3, 8, 16, 12.0), None)], mult=0.7)
    folder = write_folder(str(tmp_path / "state"), cfg, make_weights(cfg, 2))
    reqs = {f"r{i}": random_prompt(97, n, i) for i, n in enumerate((40, 3, 65, 21, 30))}
    want = plain_logits(folder, reqs)
    for steps in (trace_whole(reqs), trace_portions(reqs, seed=3), trace_mixed(reqs, max_tokens=256, seed=9)):
        runner = _runner(folder, 16, 256)
        assert not runner.cache.groups
        got = collect(steps, _replay(runner, steps))
        for rid in reqs:
            err, row, scale = max_error(got[rid], want[rid])
            assert err <= 2e-5 * scale, (rid, err, row)
        assert not runner.cache.live()
    prompts = [random_prompt(97, n, 40 + n) for n in (5, 17, 9)]
    eng = LLMEngine.from_folder(folder, dtype="float32", device="cpu", max_model_len=64, page_size=16, num_kv_blocks=0, max_num_seqs=2,
                                max_num_batched_tokens=24, ops=CpuOps())
    got = eng.generate(prompts, SamplingParams(max_tokens=6, ignore_eos=True))
    assert [r.token_ids for r in got] == [plain_greedy(folder, p, 6) for p in prompts]


def test_a_request_that_the_blocks_pages_cannot_hold_is_refused(folders):
    eng = LLMEngine.from_folder(folders["A"], dtype="float32", device="cpu", max_model_len=1024, page_size=16, num_kv_blocks=8,
                                max_num_seqs=1, max_num_batched_tokens=64, ops=CpuOps())
    assert eng.runner.cache.pages_per_group()[1] == 3                # 3 pages of blocks: 192 positions
    eng.add_request(random_prompt(160, 150, 1), SamplingParams(max_tokens=42, ignore_eos=True))
    with pytest.raises(ValueError, match="page"):
        eng.add_request(random_prompt(160, 150, 1), SamplingParams(max_tokens=60, ignore_eos=True))


# ------------------------------------------------------ the plain implementation itself ---
def test_plain_mechanisms_by_hand():
    """The plain implementation's own small facts, so that an oracle that is wrong in the same way as
    the engine does not go unnoticed."""
    P = plain_kosusun
    assert torch.allclose(P.unit_rms(torch.tensor([[3.0, 4.0, 0.0, 0.0]], dtype=F64), 2.75),
                          torch.tensor([[1.0, 4.0 / 3.0, 0.0, 0.0]], dtype=F64))       # eps inside the root: sqrt(6.25 + 2.75)
    # base 1: every frequency is 1, over the factor 2: an angle of 1 at position 2; element 4 passes
    z = torch.zeros(3, 5, dtype=F64)
    z[2] = torch.tensor([1.0, 0.0, 0.0, 2.0, 9.0])
    c, s = math.cos(1.0), math.sin(1.0)
    rot = {"dims": 4, "base": 1.0, "scaling": {"factor": 2.0}}
    assert torch.allclose(P.turn(z, torch.arange(3), rot, False)[2], torch.tensor([c, -2 * s, s, 2 * c, 9.0], dtype=F64))
    assert torch.allclose(P.turn(z, torch.arange(3), rot, True)[2], torch.tensor([c, s, -2 * s, 2 * c, 9.0], dtype=F64))
    r = P.turn(torch.tensor([[0.0, 1.0, 0.0, 0.0]], dtype=F64), torch.tensor([3]), {"dims": 4, "base": 100.0}, False)
    assert torch.allclose(r[0], torch.tensor([0.0, math.cos(0.3), 0.0, math.sin(0.3)], dtype=F64))
    # a window of 4 and blocks of 3 at position 9: tokens 6..9, blocks that end at or before 5; at 8 block 1 is not seen yet
    assert P.seen_tokens(9, 4) == [6, 7, 8, 9] and P.seen_blocks(9, 4, 3) == [0, 1]
    assert P.seen_tokens(8, 4) == [5, 6, 7, 8] and P.seen_blocks(8, 4, 3) == [0]     # tokens 3 and 4 are out of sight
    assert P.seen_blocks(5, 4, 3) == [] and P.seen_blocks(6, 4, 3) == [0]
    assert P.pooled_blocks(torch.arange(8, dtype=F64).view(8, 1), 3).tolist() == [[1.0], [4.0]]
    # the sink counts once, unscaled, and has no value: two equal scores of 0 and a sink of ln 2 weigh 1/4 each
    assert torch.allclose(P.softmax_with_sink(torch.zeros(2, dtype=F64), math.log(2.0)), torch.tensor([0.25, 0.25], dtype=F64))
    assert torch.allclose(P.softmax_with_sink(torch.zeros(2, dtype=F64), None), torch.tensor([0.5, 0.5], dtype=F64))
    # tokens and blocks share one softmax: equal scores, window 1, blocks of 2: position 4 sees itself and two blocks
    v = torch.tensor([1.0, 3.0, 5.0, 7.0, 9.0], dtype=F64).view(5, 1, 1)
    o = P.windowed_attention(torch.zeros(5, 1, 1, dtype=F64), torch.zeros(5, 1, 1, dtype=F64), v, 1.0, 1, 2, None)
    assert math.isclose(float(o[4, 0, 0]), (2.0 + 6.0 + 9.0) / 3) and math.isclose(float(o[3, 0, 0]), (2.0 + 7.0) / 2)
    # retention's memory: decay 1/2, k = v = q = 1: S = 1, 1.5, 1.75
    one = torch.ones(3, 1, 1, dtype=F64)
    assert torch.allclose(P.decaying_memory(one, one, one, [0.5]).flatten(), torch.tensor([1.0, 1.5, 1.75], dtype=F64))
    # the matrix memory: log forget gate 0, log input gate -1: m stays 0, S = n = e^-1, 2 e^-1, 3 e^-1; the floor is 1
    # until n exceeds it
    i, f = torch.full((3, 1), -1.0, dtype=F64), torch.zeros(3, 1, dtype=F64)
    n = torch.tensor([1.0, 2.0, 3.0], dtype=F64) / math.e
    assert torch.allclose(P.matrix_memory(one, one, one * 5, i, f).flatten(), 5 * n / (torch.clamp(n, min=1.0) + 1e-6))
    # m starts at 0, not at minus infinity: an input gate of -3 alone leaves exp(-3) in S and the floor at 1
    assert math.isclose(float(P.matrix_memory(one[:1], one[:1], one[:1], i[:1] * 3, f[:1])), math.exp(-3.0) / (1.0 + 1e-6))
    # an input gate above the running maximum takes it over: S is rescaled, the floor falls to exp(-2)
    i = torch.tensor([[0.0], [2.0]], dtype=F64)
    s1 = math.exp(-2.0) + 1.0
    assert math.isclose(float(P.matrix_memory(one[:2], one[:2], one[:2], i, f[:2])[1]), s1 / (s1 + 1e-6))
    assert math.isclose(float(P.gelu_tanh(torch.tensor(1.0, dtype=F64))), 0.5 * (1 + math.tanh(math.sqrt(2 / math.pi) * 1.044715)))
    # one layer without feed-forward whose mixer gives nothing: the scaled embedding stands, the logits are scaled
    cfg = _config(3, 2, [_layer("parallel", _parallel(_window(1, 1, 2, 1, 2, 2, _rot(2)), _retention(1, 2, 1, [0.5], _rot(2))), None)],
                  embed=3.0, logit=0.25)
    w = {k: v.to(F64) for k, v in make_weights(cfg, 1).items()}
    w["l0.mix.left.o"].zero_(), w["l0.mix.right.o"].zero_()
    res = []
    logits = plain_kosusun.forward(cfg, w, [2, 1], res)
    assert torch.allclose(res[0], 3.0 * w["embed"][[2, 1]])
    assert torch.allclose(logits, 0.25 * plain_kosusun.weighted_norm(res[0], w["final.norm"], 1e-5) @ w["head"].T)
