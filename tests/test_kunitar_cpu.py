"""Kunitar through the engine's own logic on the CPU (the kernel library replaced by the plain-torch
stand-in of tests/cpu_ops.py): configuration and weights, layers that read another layer's vectors
over windows of their own, state slots, all ways of cutting the work, pages and slots that change
hands, and greedy generation through the scheduler, against the plain implementation; and the plain
implementation's own facts by hand."""
import json
import math

import numpy as np
import pytest
import torch

import plain_kunitar
from cpu_ops import CpuOps
from helpers import collect, max_error, random_prompt, trace_mixed, trace_portions, trace_prefill_then_decode, trace_whole
from kunitar_helpers import (SMALL, L, W, _config, _dense, _latent, _layer, _moe, _wkv, make_folder, make_weights, plain_greedy,
                             plain_logits, write_folder)
from tiny_llm_infer_amd.config import ConfigError, KunitarConfig
from tiny_llm_infer_amd.engine.llm_engine import LLMEngine
from tiny_llm_infer_amd.engine.loading import load_model, random_model, write_random_model
from tiny_llm_infer_amd.engine.replay import Replayer
from tiny_llm_infer_amd.engine.runner import ModelRunner
from tiny_llm_infer_amd.registry import architecture_of
from tiny_llm_infer_amd.sampling.params import SamplingParams
from tiny_llm_infer_amd.weights.loader import AnySize, TensorDecl, WeightError

F64 = torch.float64


@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    root = tmp_path_factory.mktemp("kunitar")
    return {name: make_folder(str(root / name), name) for name in SMALL}


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
    from tiny_llm_infer_amd.models.kunitar import kunitar_spec
    for name, (cfg, _, _, _) in SMALL.items():
        typed = KunitarConfig.from_dict(cfg)
        assert typed.to_dict() == cfg
        assert architecture_of(cfg).name == "Kunitar"
        spec = kunitar_spec(typed)
        assert [c.block for c in spec.schedule] == list(range(len(cfg["layers"])))
        own = [i for i, layer in enumerate(cfg["layers"]) if layer["type"] == L and "kv_from" not in layer["mixer"]]
        for i, (call, layer) in enumerate(zip(spec.schedule, cfg["layers"])):
            if layer["type"] == W:
                assert call.cache == -1
            else:
                assert call.cache == own.index(layer["mixer"].get("kv_from", i)) and call.writes_cache == (i in own)
    # a cache layer keeps as much as the widest of the windows that read it
    windows = [b.mixer.params["cache_window"] for b in kunitar_spec(KunitarConfig.from_dict(SMALL["A"][0])).blocks if b.mixer.kind == L]
    assert windows == [37, 37, 37]


@pytest.mark.parametrize("change, message", [
    (lambda c: c.pop("width"), "width"),
    (lambda c: c.pop("token_side"), "dim"),
    (lambda c: c["layers"][0].update(type="conv"), "layer type"),
    (lambda c: c["layers"][0]["mixer"]["mask"].update(size=0), "size"),
    (lambda c: c["layers"][0]["mixer"]["rot"].update(dims=6), "rot.dims"),
    (lambda c: c["layers"][0]["mixer"]["rot"].update(base=0.0), "base"),
    (lambda c: c["layers"][0]["mixer"].pop("q_rank"), "q_rank"),
    (lambda c: c["layers"][0]["mixer"].pop("scale"), "scale"),
    (lambda c: c["layers"][2]["mixer"].update(kv_from=1), "kv_from"),
    (lambda c: c["layers"][2]["mixer"].update(kv_from=3), "kv_from"),
    (lambda c: c["layers"][3]["mixer"].update(kv_from=2), "kv_from"),
    (lambda c: c["layers"][2]["mixer"].update(kv_rank=16), "latent size or rotation"),
    (lambda c: c["layers"][2]["mixer"]["rot"].update(base=7.0), "latent size or rotation"),
    (lambda c: c["layers"][1]["mixer"].pop("heads"), "heads"),
    (lambda c: c["layers"][1]["mlp"]["router"].update(top=7), "cannot be chosen"),
    (lambda c: c["layers"][1]["mlp"].update(kind="glu"), "feed-forward kind"),
    (lambda c: c["norm"].update(eps=0.0), "eps"),
])
def test_config_errors(change, message):
    cfg = json.loads(json.dumps(SMALL["A"][0]))
    change(cfg)
    with pytest.raises(ConfigError, match=message):
        KunitarConfig.from_dict(cfg)


def test_a_checkpoint_that_does_not_fit_is_refused(tmp_path):
    cfg, rank, _, seed = SMALL["A"]
    w = make_weights(cfg, rank, seed)
    del w["l0.mix.dq.norm"]
    w["l1.mix.u"] = w["l1.mix.u"][:-1].contiguous()
    w["l2.mix.dkv"] = w["l0.mix.dkv"].clone()                  # a layer that reads another's vectors has no matrix for its own
    w["head"] = w["embed"].clone()
    folder = write_folder(str(tmp_path / "bad"), cfg, w)
    with pytest.raises(WeightError) as err:
        load_model(folder, "float32", "cpu", ops=CpuOps())
    assert err.value.missing == ["l0.mix.dq.norm"] and err.value.unexpected == ["head", "l2.mix.dkv"]
    assert [n for n, _, _ in err.value.wrong_shape] == ["l1.mix.u"]


def test_the_checkpoint_says_the_decays_inner_size(tmp_path):
    """No key of the configuration gives it; matrices that do not meet are refused."""
    cfg, _, _, seed = SMALL["B"]
    for rank in (1, 3, 40):
        model, _ = load_model(write_folder(str(tmp_path / f"r{rank}"), cfg, make_weights(cfg, rank, seed)), "float32", "cpu", ops=CpuOps())
        assert model.blocks[0].mixer.rank == rank
    w = make_weights(cfg, 6, seed)
    w["l0.mix.w2"] = w["l0.mix.w2"][:, :5].contiguous()
    with pytest.raises(ValueError, match="meet in 6 and 5"):
        load_model(write_folder(str(tmp_path / "odd"), cfg, w), "float32", "cpu", ops=CpuOps())
    assert AnySize(7) == 7 and TensorDecl("x", (AnySize(7), 2)).shape == (7, 2)


def test_random_weights_load_and_generate(tmp_path):
    cfg = json.loads(json.dumps(SMALL["A"][0]))
    cfg["layers"][1]["mixer"]["decay_rank"] = 11
    typed = KunitarConfig.from_dict(cfg)
    assert typed.to_dict() == cfg
    folder = write_random_model(str(tmp_path / "random"), "Kunitar", typed, 3)
    eng = LLMEngine.from_folder(folder, dtype="float32", device="cpu", max_model_len=64, page_size=16, num_kv_blocks=16, max_num_seqs=2,
                                max_num_batched_tokens=32, ops=CpuOps())
    assert eng.runner.model.blocks[1].mixer.rank == 11
    assert len(eng.generate([[1, 2, 3]], SamplingParams(max_tokens=4, ignore_eos=True))[0].token_ids) == 4


# ---------------------------------------------------------------- cache and state ---
def test_groups_and_slots(folders):
    runner = _runner(folders["A"], 16, 256)
    (group,) = runner.cache.groups
    assert group.need.window == 37 and group.cache_layers == [0]
    assert tuple(runner.group_tensors[0]["latent"].shape[2:]) == (16, 32 + 8)
    states = [s for s in runner.states if s is not None]
    assert [set(s) for s in states] == [{"S", "last"}]
    assert tuple(states[0]["S"].shape) == (5, 3, 16, 16) and tuple(states[0]["last"].shape) == (5, 64)
    runner = _runner(folders["R"], 32, 256)
    assert [g.need.window for g in runner.cache.groups] == [65]


def test_the_group_gives_pages_back_behind_the_widest_window(folders):
    folder = folders["A"]
    reqs = _requests("A", [150], seed=2)
    want = plain_logits(folder, reqs)
    runner = _runner(folder, 16, 160)
    steps = trace_prefill_then_decode(reqs, tail=60)[:-1]
    got = collect(steps, _replay(runner, steps))
    (table,) = runner.cache.get("r0").tables
    held = [b for b, p in enumerate(table) if p >= 0]
    assert held == list(range((149 - 36) // 16, 10))            # the next row is at 149 and reads 36 back
    err, row, scale = max_error(got["r0"], want["r0"][:-1])
    assert err <= 2e-5 * scale, (err, row)


# ------------------------------------------------------------------ all the cuts ---
@pytest.mark.parametrize("name", list(SMALL))
def test_all_cuts_match_plain(folders, name):
    folder = folders[name]
    reqs = _requests(name, [70, 45, 83, 33, 1, 58, 2], seed=5)
    want = plain_logits(folder, reqs)
    max_tokens = 256
    cuts = {
        "whole": trace_whole(reqs),
        "decode": trace_prefill_then_decode(reqs),
        "portions": trace_portions(reqs, seed=3),
        "mixed": trace_mixed(reqs, max_tokens=max_tokens, seed=9),
    }
    for cut, steps in cuts.items():
        runner = _runner(folder, SMALL[name][2], max_tokens)
        got = collect(steps, _replay(runner, steps))
        for rid in reqs:
            err, row, scale = max_error(got[rid], want[rid])
            assert err <= 3e-5 * max(1.0, scale), f"{name}/{cut}/{rid}: error {err} at token {row}"
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
        runner = _runner(folder, SMALL[name][2], 64)
        got = collect(steps, _replay(runner, steps))
        err, row, scale = max_error(got["r0"], want["r0"])
        assert err <= 3e-5 * scale, (name, err, row)


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
        for t in (s or {}).values():
            t.fill_(-5.0)
    steps = trace_portions(reqs, seed=1)
    got = collect(steps, _replay(runner, steps))
    for rid in reqs:
        err, row, scale = max_error(got[rid], want[rid])
        assert err <= 3e-5 * scale, (rid, err, row)
    assert runner.cache.pages_taken_total > runner.cache.num_pages


def test_unequal_requests_together_equal_each_alone(folders):
    folder = folders["S"]
    reqs = _requests("S", [3, 100, 34, 65], seed=60)
    alone = {}
    for rid, toks in reqs.items():
        runner = _runner(folder, 16, 256)
        alone[rid] = _replay(runner, trace_whole({rid: toks}))[0]
    runner = _runner(folder, 16, 512)
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
    args = dict(dtype="float32", device="cpu", max_model_len=128, page_size=SMALL[name][2], num_kv_blocks=64,
                max_num_seqs=4, max_num_batched_tokens=24, ops=CpuOps())
    eng = LLMEngine.from_folder(folder, **args)
    got = eng.generate(prompts, SamplingParams(max_tokens=12, ignore_eos=True))
    assert [r.token_ids for r in got] == want
    eng.runner.cache.check()
    assert eng.runner.cache.free_pages() == eng.runner.cache.pages_per_group()


def test_a_model_that_keeps_state_only(tmp_path):
    """Recurrent layers alone: no group of pages at all, requests live by their slots."""
    cfg = _config(97, 40, 6, [_layer(W, _wkv(2, 12), _dense(33)), _layer(W, _wkv(3, 8), None)])
    folder = write_folder(str(tmp_path / "state"), cfg, make_weights(cfg, 4, 2))
    reqs = {f"r{i}": random_prompt(97, n, i) for i, n in enumerate((40, 3, 65, 21, 30))}
    want = plain_logits(folder, reqs)
    for steps in (trace_whole(reqs), trace_mixed(reqs, max_tokens=256, seed=9)):
        runner = _runner(folder, 16, 256)
        assert not runner.cache.groups
        got = collect(steps, _replay(runner, steps))
        for rid in reqs:
            err, row, scale = max_error(got[rid], want[rid])
            assert err <= 3e-5 * scale, (rid, err, row)
        assert not runner.cache.live()


def test_blocks_of_another_arrangement_are_refused():
    from tiny_llm_infer_amd.models.kunitar import kunitar_spec
    from tiny_llm_infer_amd.parts.base import build_part
    from tiny_llm_infer_amd.engine.model import Model
    block = Model(kunitar_spec(KunitarConfig.from_dict(SMALL["C"][0]))).blocks[0]
    with pytest.raises(TypeError, match="another kind"):
        block.forward(torch.zeros(1, 72), torch.zeros(1, 72), None)
    with pytest.raises(ValueError, match="on its input"):
        build_part("ffn", _experts_spec(gated=True, weight_on="input", activation="silu"))


def _experts_spec(**params):
    from tiny_llm_infer_amd.config.base import PartSpec
    return PartSpec("routed_experts", {"hidden_size": 8, "experts": 2, "top": 1, "intermediate_size": 8, **params},
                    {"router": "r", "experts": "e{}."})


# ------------------------------------------------------ the plain implementation itself ---
def test_plain_mechanisms_by_hand():
    """The plain implementation's own small facts, so that an oracle that is wrong in the same way as
    the engine does not go unnoticed."""
    P = plain_kunitar
    assert torch.allclose(P.unit_rms(torch.tensor([[3.0, 4.0, 0.0, 0.0]], dtype=F64), 2.75),
                          torch.tensor([[1.0, 4.0 / 3.0, 0.0, 0.0]], dtype=F64))       # eps inside the root: sqrt(6.25 + 2.75)
    # neighbours turn together; base 100: the second pair's frequency is 1/10
    z = torch.zeros(4, 5, dtype=F64)
    z[3] = torch.tensor([1.0, 0.0, 0.0, 2.0, 9.0])
    r = P.turn(z, torch.arange(4), 4, 100.0)[3]
    assert torch.allclose(r, torch.tensor([math.cos(3.0), math.sin(3.0), -2 * math.sin(0.3), 2 * math.cos(0.3), 9.0], dtype=F64))
    assert P.seen(9, 4) == [6, 7, 8, 9] and P.seen(2, 4) == [0, 1, 2] and P.seen(5, 1) == [5]
    # equal scores over a window of two: the mean of two values
    v = torch.tensor([1.0, 3.0, 5.0], dtype=F64).view(3, 1, 1)
    assert P.windowed(torch.zeros(3, 1, 1, dtype=F64), torch.zeros(3, 1, 1, dtype=F64), v, 1.0, 2).flatten().tolist() == [1.0, 2.0, 4.0]
    # decays 1/2, r = k = v = 1, bonus 3: what the token adds itself counts three times, and is in the state for the next
    one = torch.ones(3, 1, 1, dtype=F64)
    o = P.decayed_memory(one, one, one, one * 0.5, torch.full((1, 1), 3.0, dtype=F64))
    assert torch.allclose(o.flatten(), torch.tensor([3.0, 4.0, 4.5], dtype=F64))        # S: 0, 1, 1.5
    # a decay a channel: only the channel that r reads matters
    k, d = torch.tensor([[[1.0, 1.0]]] * 2, dtype=F64), torch.tensor([[[0.1, 0.7]]] * 2, dtype=F64)
    k3, d3, r3 = (torch.cat([t, t[:1]]) for t in (k, d, torch.tensor([[[0.0, 1.0]]] * 2, dtype=F64)))
    assert torch.allclose(P.decayed_memory(r3, k3, one, d3, torch.zeros(1, 2, dtype=F64)).flatten(), torch.tensor([0.0, 1.0, 1.7], dtype=F64))
    assert P.shifted(torch.tensor([[1.0], [2.0], [3.0]], dtype=F64)).flatten().tolist() == [0.0, 1.0, 2.0]
    w = {"w1": torch.zeros(1, 2, dtype=F64), "w2": torch.zeros(3, 1, dtype=F64), "w0": torch.tensor([0.0, 1.0, -50.0], dtype=F64)}
    assert torch.allclose(P.decays(torch.ones(1, 2, dtype=F64), w, ""), torch.tensor([[math.exp(-1), math.exp(-math.e), 1.0]], dtype=F64))
    assert math.isclose(float(P.gelu_erf(torch.tensor(1.0, dtype=F64))), 0.5 * (1 + math.erf(math.sqrt(0.5))))
    assert math.isclose(float(P.gelu_tanh(torch.tensor(1.0, dtype=F64))), 0.5 * (1 + math.tanh(math.sqrt(2 / math.pi) * 1.044715)))
    assert P.squared_relu(torch.tensor([-2.0, 3.0], dtype=F64)).tolist() == [0.0, 9.0]
    # the weight goes on the expert's input: it counts twice in the square; the best of two by its score alone
    w = {"router": torch.tensor([[0.0], [math.log(3.0)]], dtype=F64)}
    for e, s in ((0, 5.0), (1, 2.0)):
        w[f"e{e}.up"], w[f"e{e}.down"] = torch.ones(1, 1, dtype=F64), torch.full((1, 1), s, dtype=F64)
    y = P.experts(torch.ones(1, 1, dtype=F64), {"router": {"top": 1}, "shared": None}, w, "")
    assert math.isclose(float(y), 0.75 ** 2 * 2.0)
    y = P.experts(torch.ones(1, 1, dtype=F64), {"router": {"top": 2}, "shared": None}, w, "")
    assert math.isclose(float(y), 0.75 ** 2 * 2.0 + 0.25 * 5.0)
    # one layer whose sublayers give nothing and whose side does: the scaled embedding, and the side's normed row behind it
    cfg = _config(3, 2, 1, [_layer(W, _wkv(1, 2), None)], embed=3.0)
    w = {k: t.to(F64) for k, t in make_weights(cfg, 1, 1).items()}
    w["l0.mix.o"].zero_()
    w["l0.side.proj"] = torch.tensor([[2.0], [0.0]], dtype=F64)
    res = []
    logits = P.forward(cfg, w, [2, 1], res)
    x = 3.0 * w["embed"][[2, 1]]
    g = P.gelu_tanh(x @ w["l0.side.gate"].T) * w["side.embed"][[2, 1]]
    y = torch.cat([2 * g, 0 * g], dim=1)
    assert torch.allclose(res[0], x + y / torch.sqrt(2 * g * g + 1e-5) * w["l0.side.norm"])
    assert torch.allclose(logits, P.weighted_norm(res[0], w["final.norm"], 1e-5) @ w["embed"].T)
