"""Kunitar on the GPU: each mechanism's kernels alone against the plain implementation's function for it
(the recurrence over portions and slots that change hands, keys just inside and outside a window, mixes
with kept rows, stacked products, experts without a gate, a token's own vector), then the model through
the step function in every cut, in float32 and in bfloat16, long decoding through recorded launches, and
greedy generation through the engine and the command line."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

import plain_kunitar
from helpers import collect, max_error, random_prompt, trace_mixed, trace_portions, trace_prefill_then_decode, trace_whole
from kunitar_helpers import (SMALL, L, W, _config, _dense, _latent, _layer, _moe, _wkv, make_folder, make_weights, plain_greedy,
                             plain_logits, write_folder)

pytestmark = pytest.mark.gpu
F64 = torch.float64
# of the largest logit
TOL = {"float32": 3e-5, "bfloat16": 5e-2}
DTYPES = {"float32": torch.float32, "bfloat16": torch.bfloat16}


@pytest.fixture(scope="module")
def ops():
    from tiny_llm_infer_amd.kernels.ops import HipOps
    return HipOps("cuda:0")


@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    root = tmp_path_factory.mktemp("kunitar")
    return {name: make_folder(str(root / name), name) for name in SMALL}


@pytest.fixture(scope="module")
def clear_folders(tmp_path_factory):
    """Weights without close calls of a router and with scores that do not multiply rounding (for bfloat16)."""
    root = tmp_path_factory.mktemp("kunitar_clear")
    return {name: make_folder(str(root / name), name, clear=True) for name in SMALL}


def _runner(folder, dtype, max_tokens, page, max_requests=4):
    from tiny_llm_infer_amd.engine.loading import load_model
    from tiny_llm_infer_amd.engine.runner import ModelRunner
    model, _ = load_model(folder, dtype, "cuda:0", max_model_len=2048)
    return ModelRunner(model, model.env, page_size=page, num_pages=max_tokens // page,
                       max_requests=max_requests, max_batch_tokens=1024)


def _replay(runner, steps):
    from tiny_llm_infer_amd.engine.replay import Replayer
    rp = Replayer(runner)
    return {st["step"]: rp.run_step(st) for st in steps}


def _requests(vocab, lengths, seed):
    return {f"r{i}": random_prompt(vocab, n, seed + i) for i, n in enumerate(lengths)}


def _close(got, want, tol, what):
    got, want = got.detach().double().cpu(), want.double()
    err, scale = float((got - want).abs().max()), float(want.abs().max())
    assert err <= tol * max(scale, 1e-6), f"{what}: error {err:.3e}, scale {scale:.3e}"


def _all_cuts(folder, dtype, reqs, want, page, max_tokens, tol, what):
    cuts = {
        "whole": trace_whole(reqs),
        "decode": trace_prefill_then_decode(reqs),
        "portions": trace_portions(reqs, seed=3),
        "mixed": trace_mixed(reqs, max_tokens=max_tokens, seed=9),
    }
    for cut, steps in cuts.items():
        runner = _runner(folder, dtype, max_tokens, page)
        got = collect(steps, _replay(runner, steps))
        for rid in reqs:
            err, row, scale = max_error(got[rid], want[rid])
            assert err <= tol * scale, f"{what}/{dtype}/{cut}/{rid}: error {err:.3e} at token {row} (scale {scale:.3e})"
        runner.cache.check()
        assert not runner.cache.live() and runner.cache.free_pages() == runner.cache.pages_per_group()


def _view(starts, counts, slots):
    """A step of sequences that stand at ``starts`` and bring ``counts`` rows, as the step function packs it."""
    from tiny_llm_infer_amd.parts.base import StepView
    i32 = lambda v: torch.tensor([int(x) for x in v], dtype=torch.int32, device="cuda")
    row_start = [0] + list(np.cumsum(counts))
    pos = [s + j for s, c in zip(starts, counts) for j in range(c)]
    sor = [i for i, c in enumerate(counts) for _ in range(c)]
    totals = [s + c for s, c in zip(starts, counts)]
    return StepView(num_rows=sum(counts), num_seqs=len(counts), token_ids=i32(pos), positions=i32(pos), seq_of_row=i32(sor),
                    row_start=i32(row_start), seq_start=i32(starts), seq_len=i32(totals), slots=i32(slots),
                    sample_rows=i32([0]), h_row_start=[int(r) for r in row_start], h_seq_start=list(starts),
                    h_seq_len=totals, h_slots=list(slots), max_rows_per_seq=max(counts), max_seq_len=max(totals),
                    reach=max(128, 1 << (max(totals) - 1).bit_length()))


def _portions(lengths, cuts):
    """Steps (starts, counts, which sequences) that bring sequences of these lengths side by side in portions of ``cuts`` rows."""
    at, k = [0] * len(lengths), 0
    while any(a < n for a, n in zip(at, lengths)):
        live = [i for i in range(len(lengths)) if at[i] < lengths[i]]
        counts = [min(cuts[(k + i) % len(cuts)], lengths[i] - at[i]) for i in live]
        yield [at[i] for i in live], counts, live
        for i, c in zip(live, counts):
            at[i] += c
        k += 1


# ------------------------------------------------------------- the recurrence, alone ---
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("lengths, cuts", [([61, 97, 45], [1, 43, 2, 16, 33, 7]), ([700, 30, 301], [530, 190, 1, 2, 64]), ([24, 20, 3], [1]),
                                           ([130, 129, 64], [64, 65, 128])])
@pytest.mark.parametrize("heads, dk, dv, rank", [(3, 16, 16, 8), (2, 64, 64, 32), (1, 128, 128, 64), (2, 48, 80, 20), (3, 20, 12, 5), (1, 7, 30, 3),
                                                 (2, 200, 16, 12), (5, 32, 64, 132)])
@pytest.mark.parametrize("chunks", [True, False], ids=["chunks", "rows"])
def test_the_recurrence_in_portions_and_slots_that_are_used_again(ops, dtype, heads, dk, dv, rank, lengths, cuts, chunks, monkeypatch):
    """Three sequences side by side through the recurrence, in portions of all sizes, twice with their slots exchanged; channels
    that keep everything, that forget within a row and all between."""
    if chunks and (dtype == "float32" or not ops.lib.tli_wkv_chunked_takes(dk, dv, rank)):
        pytest.skip("these rows do not go through chunks")
    monkeypatch.setattr(ops, "recurrence_in_chunks", chunks)
    if max(lengths) > 500 and dk > 128:
        lengths = [min(n, 300) for n in lengths]
    g = torch.Generator().manual_seed(dk + dv + rank)
    dt = DTYPES[dtype]
    w0 = torch.randn(heads * dk, generator=g) * 2.0 - 2.0
    w0[0], w0[1], w0[2] = -30.0, 3.0, 6.0                            # decays of 1, of 2e-9, of 0
    w2 = (torch.randn(heads * dk, rank, generator=g) * rank ** -0.5).to(dt)
    u = torch.randn(heads, dk, generator=g) * 0.4 + 0.7
    weight = torch.randn(heads * dv, generator=g) * 0.2 + 1.0
    state = torch.full((3, *ops.wkv_state_shape(heads, dk, dv)), 7.0, device="cuda")          # what another request left
    at = [0, heads * dk, 2 * heads * dk, 2 * heads * dk + heads * dv, 2 * heads * dk + 2 * heads * dv]
    for slots in ([0, 1, 2], [2, 0, 1]):
        proj = [torch.randn(n, at[4], generator=g) for n in lengths]
        for p in proj:
            p[:, at[1]:at[2]] += p[:, :at[1]]                                                  # (no output that is all rounding)
        proj = [p.to(dt) for p in proj]
        z = [torch.randn(n, rank, generator=g) * 1.5 for n in lengths]
        got = [[] for _ in lengths]
        for k, (starts, counts, live) in enumerate(_portions(lengths, cuts)):
            rows = torch.cat([proj[i][s:s + c] for i, s, c in zip(live, starts, counts)]).cuda()
            inner = torch.cat([z[i][s:s + c] for i, s, c in zip(live, starts, counts)]).cuda()
            strides = (rank, 1)
            if k % 2:                                                                          # both orders of the inner rows
                inner, strides = inner.t().contiguous(), (1, len(rows))
            y = ops.wkv(rows, inner, strides, w2.cuda(), w0.cuda(), u.cuda(), state, _view(starts, counts, [slots[i] for i in live]),
                        heads, dk, dv, weight.cuda(), 1e-5, dt)
            r = 0
            for i, c in zip(live, counts):
                got[i].append(y[r:r + c].cpu())
                r += c
        for i, n in enumerate(lengths):
            r, key, v, gate = (proj[i][:, a:b].double() for a, b in zip(at, at[1:]))
            d = torch.exp(-torch.exp(torch.tanh(z[i].double()) @ w2.double().T + w0.double())).view(n, heads, dk)
            o = plain_kunitar.decayed_memory(r.view(n, heads, dk), key.view(n, heads, dk), v.view(n, heads, dv), d, u.double())
            want = plain_kunitar.unit_rms(o, 1e-5).reshape(n, heads * dv) * weight.double() * torch.nn.functional.silu(gate)
            _close(torch.cat(got[i]), want, 1e-4 if dtype == "float32" else 1.5e-2, f"sequence {i} in slot {slots[i]}")


@pytest.mark.parametrize("dk, dv", [(64, 64), (128, 128), (32, 48)])
def test_chunks_give_the_states_of_the_recurrence_row_by_row(ops, dk, dv):
    """The state behind a portion, float32 and not normed: chunks against rows, to float32's own precision, also behind
    portions that end at a chunk's edge and past it, and with decays whose product over a chunk is far below float32's range."""
    g = torch.Generator().manual_seed(dk)
    heads, rank = 2, 16
    for lengths in ([64, 130, 1], [300, 15, 63]):
        T = sum(lengths)
        proj = torch.randn(T, 2 * heads * (dk + dv), generator=g).to(torch.bfloat16).cuda()
        z = torch.randn(T, rank, generator=g).cuda()
        w2 = (torch.randn(heads * dk, rank, generator=g) * 0.5).to(torch.bfloat16).cuda()
        w0 = torch.linspace(-9.0, 3.0, heads * dk).cuda()
        u, weight = torch.ones(heads, dk).cuda(), torch.ones(heads * dv).cuda()
        states = []
        for chunks in (True, False):
            ops.recurrence_in_chunks = chunks
            try:
                state = torch.randn(3, heads, dv, dk, generator=torch.Generator().manual_seed(5)).cuda()
                ops.wkv(proj, z, (rank, 1), w2, w0, u, state, _view([0, 40, 7], lengths, [2, 0, 1]), heads, dk, dv, weight, 1e-5, torch.bfloat16)
            finally:
                ops.recurrence_in_chunks = True
            states.append(state)
        _close(states[0], states[1].cpu(), 2e-5, f"{lengths}")


# ------------------------------------------------ norms and mixes with the row before ---
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("n", [64, 100, 2048, 4104])
def test_norms_and_mixes_in_portions(ops, dtype, n):
    """x += w1 unit(y), h = w2 unit(x), mixes of h with the row before it: in one pass for single rows, in two for portions,
    through slots that are used again; the row before position 0 is zeros."""
    g = torch.Generator().manual_seed(n)
    dt, eps = DTYPES[dtype], 1e-5
    mu = torch.randn(5, n, generator=g) * 0.5 + 0.4
    w1, w2 = torch.randn(n, generator=g), torch.randn(n, generator=g) * 0.2 + 1.0
    kept = torch.full((3, n), 9.0, dtype=dt, device="cuda")
    lengths, P = [9, 14, 5], plain_kunitar
    for slots, cuts in (([0, 1, 2], [1]), ([2, 0, 1], [3, 1, 5, 2]), ([1, 2, 0], [1, 4])):
        x0 = [torch.randn(c, n, generator=g) for c in lengths]
        y = [torch.randn(c, n, generator=g).to(dt) for c in lengths]
        got = [[] for _ in lengths]
        for starts, counts, live in _portions(lengths, cuts):
            step = _view(starts, counts, [slots[i] for i in live])
            take = lambda t: torch.cat([t[i][s:s + c] for i, s, c in zip(live, starts, counts)]).cuda().contiguous()
            resid, delta = take(x0), take(y)
            mixed = ops.norm_add_norm_mixes(resid, delta, w1.cuda(), eps, w2.cuda(), eps, dt, (mu.cuda(), kept), step)
            assert (mixed is not None) == (max(counts) == 1)
            if mixed is None:
                mixed = ops.token_mixes(ops.norm_add_norm(resid, delta, w1.cuda(), eps, w2.cuda(), eps, dt), mu.cuda(), kept, step)
            want = take(x0).cpu().double() + P.weighted_norm(take(y).cpu().double(), w1.double(), eps)
            _close(resid, want, 1e-5, "the residual")
            r = 0
            for i, c in zip(live, counts):
                got[i].append(mixed[:, r:r + c].cpu())
                r += c
        for i in range(len(lengths)):
            h = P.weighted_norm(x0[i].double() + P.weighted_norm(y[i].double(), w1.double(), eps), w2.double(), eps)
            want = torch.stack([h + (P.shifted(h) - h) * mu[m].double() for m in range(5)])
            _close(torch.cat(got[i], dim=1), want, 2e-5 if dtype == "float32" else 1.5e-2, f"sequence {i}")


def test_norms_of_a_products_partial_sums_and_of_wanted_rows(ops):
    from tiny_llm_infer_amd.kernels.ops import DeferredSum
    g = torch.Generator().manual_seed(1)
    n, T = 192, 7
    parts = torch.randn(3, T, n, generator=g)
    w1, w2, x = torch.randn(n, generator=g), torch.randn(n, generator=g), torch.randn(T, n, generator=g)
    P = plain_kunitar
    want = x.double() + P.weighted_norm(parts.double().sum(0), w1.double(), 1e-5)
    for call in ("norm_add_norm", "norm_add"):
        resid = x.cuda()
        owed = DeferredSum(parts.cuda(), torch.bfloat16)
        if call == "norm_add":
            rows, expect = ops.norm_add(resid, owed, w1.cuda(), 1e-5, torch.bfloat16), want
        else:
            rows = ops.norm_add_norm(resid, owed, w1.cuda(), 1e-5, w2.cuda(), 1e-5, torch.bfloat16)
            expect = P.weighted_norm(want, w2.double(), 1e-5)
        _close(resid, want, 1e-2, call)
        _close(rows, expect, 1.5e-2, call)
    resid = x.cuda()
    some = torch.tensor([5, 0, 6, 1], dtype=torch.int32, device="cuda")
    y = parts[0].to(torch.bfloat16)
    got = ops.norm_add_norm(resid, y.cuda(), w1.cuda(), 1e-5, w2.cuda(), 1e-5, torch.bfloat16, rows=some, num_rows=3)
    full = P.weighted_norm(x.double() + P.weighted_norm(y.double(), w1.double(), 1e-5), w2.double(), 1e-5)
    _close(got, full[[5, 0, 6]], 1.5e-2, "wanted rows")
    assert torch.equal(resid.cpu(), x)
    _close(ops.norm_add_norm(resid, None, None, 0.0, w2.cuda(), 1e-5, torch.float32), P.weighted_norm(x.double(), w2.double(), 1e-5), 1e-5, "no delta")


# ---------------------------------------------- several inputs, several matrices, one launch ---
@pytest.mark.parametrize("rows", [1, 8, 16, 17, 64, 100, 129, 300, 1000])
@pytest.mark.parametrize("size, n, few", [(128, 96, 16), (256, 192, 24), (512, 256, 64), (1024, 640, 40), (48, 72, 5)])
def test_products_of_several_inputs(ops, rows, size, n, few):
    from tiny_llm_infer_amd.parts.base import BuildEnv
    from tiny_llm_infer_amd.parts.linear import GroupedMatrix
    g = torch.Generator().manual_seed(rows + size)
    env = BuildEnv(dtype=torch.bfloat16, device=torch.device("cuda:0"), ops=ops, max_model_len=128)
    mats = [(torch.randn(size, n, generator=g) * n ** -0.5).to(torch.bfloat16) for _ in range(4)]
    last = (torch.randn(few, n, generator=g) * n ** -0.5).to(torch.bfloat16)
    xs = torch.randn(5, rows, n, generator=g).to(torch.bfloat16)
    gm = GroupedMatrix([m.cuda() for m in mats], env, few=last.cuda())
    assert (gm.stacked is not None) == (size % 128 == 0)
    want = torch.cat([xs[i].double() @ m.double().T for i, m in enumerate(mats)], dim=1)
    for single in (False, True):
        step = _view([3] * rows, [1] * rows, list(range(rows))) if single else _view([0], [max(rows, 2)], [0])
        proj, z, (z_row, z_col) = ops.linear_groups(xs.cuda(), gm, step)
        _close(proj[:, :4 * size], want, 1e-2, f"single {single}")
        inner = z.t() if tuple(z.shape) != (rows, few) or (rows == few and z_row == 1) else z
        _close(inner, xs[4].double() @ last.double().T, 2e-5, f"few rows, single {single}")
    ops.grouped_products = False
    try:
        proj, _, _ = ops.linear_groups(xs.cuda(), gm)
    finally:
        ops.grouped_products = True
    _close(proj, want, 1e-2, "one by one")


@pytest.mark.parametrize("rows", [1, 16, 17, 100, 200, 700])
@pytest.mark.parametrize("n, out", [(128, 96), (1024, 64), (256, 3072), (100, 37)])
@pytest.mark.parametrize("act", ["gelu", "gelu_tanh", "relu2"])
def test_activations_and_tokens_vectors_where_sums_are_written(ops, rows, n, out, act):
    from tiny_llm_infer_amd.parts.base import BuildEnv
    from tiny_llm_infer_amd.parts.linear import as_matrix
    g = torch.Generator().manual_seed(rows + n)
    fn = {"gelu": plain_kunitar.gelu_erf, "gelu_tanh": plain_kunitar.gelu_tanh, "relu2": plain_kunitar.squared_relu}[act]
    for dt, tol in ((torch.bfloat16, 1e-2), (torch.float32, 3e-6)):
        env = BuildEnv(dtype=dt, device=torch.device("cuda:0"), ops=ops, max_model_len=128)
        x, w = torch.randn(rows, n, generator=g).to(dt), (torch.randn(out, n, generator=g) * 2 * n ** -0.5).to(dt)
        table, ids = torch.randn(11, 3 * out, generator=g).to(dt), torch.randint(0, 11, (rows,), generator=g).to(torch.int32)
        m = as_matrix(w.cuda(), env)
        want = fn(x.double() @ w.double().T)
        own = table.double()[ids.long(), out:2 * out]
        for separate in (False, True):
            ops.separate_activations = separate
            try:
                _close(ops.linear_act(x.cuda(), m, act), want, tol, f"{dt} alone, separate {separate}")
                _close(ops.linear_act(x.cuda(), m, act, token=(table.cuda(), out, ids.cuda())), want * own, tol, f"{dt}, separate {separate}")
            finally:
                ops.separate_activations = False


# ---------------------------------------------------------------------------- the router ---
@pytest.mark.parametrize("experts, top, groups, keep", [(16, 1, 1, 1), (6, 2, 1, 1), (64, 6, 8, 3), (130, 5, 10, 2), (256, 32, 1, 1), (3, 3, 1, 1), (48, 2, 48, 2)])
@pytest.mark.parametrize("score, group_score, normalize", [("sigmoid", "top2", False), ("sigmoid", "top2", True), ("softmax", "max", False)])
@pytest.mark.parametrize("corrected, shared", [(False, True), (True, False)])
def test_a_router_in_one_launch_chooses_as_the_one_in_two(ops, experts, top, groups, keep, score, group_score, normalize, corrected, shared):
    """Small whole numbers, so that logits are exact in any order and many scores are equal: ties go to the lower index."""
    g = torch.Generator().manual_seed(experts + top)
    n = 72
    for rows in (1, 5, 128):
        x = torch.randint(-1, 2, (rows, n), generator=g).to(torch.bfloat16).cuda()
        w = (torch.randint(-1, 2, (experts + shared, n), generator=g) * 0.25).to(torch.bfloat16).cuda()
        correction = torch.randint(-2, 3, (experts,), generator=g).float().cuda() * 0.125 if corrected else None
        how = dict(score=score, group_score=group_score, normalize=normalize, correction=correction)
        ids, weights, gate = ops.router(x, w, experts, top, groups, keep, 1.5, shared, **how)
        z = (x.double() @ w.double().t()).float().contiguous()
        ids2, weights2, gate2 = ops.route_experts(z, experts, top, groups, keep, 1.5, shared, False, **how)
        assert torch.equal(ids, ids2)
        _close(weights, weights2.cpu(), 5e-6, "weights")
        if shared:
            _close(gate, gate2.cpu(), 1e-6, "gate of the shared expert")
        s = torch.sigmoid(z[:, :experts].double()) if score == "sigmoid" else torch.softmax(z[:, :experts].double(), dim=-1)
        chosen = s.gather(1, ids.long()).cpu()
        _close(weights, (chosen / (chosen.sum(-1, keepdim=True) + 1e-20) if normalize else chosen) * 1.5, 1e-5, "weights of the chosen")


# --------------------------------------------------------------- experts without a gate ---
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("rows", [1, 9, 130, 600])
@pytest.mark.parametrize("experts, top, n, ff, shared", [(6, 2, 64, 48, True), (16, 1, 128, 96, False), (3, 3, 100, 37, True), (5, 2, 256, 200, False)])
def test_experts_without_a_gate(ops, dtype, rows, experts, top, n, ff, shared):
    """The square of relu; the weight on the input (it counts twice) or on the output."""
    g = torch.Generator().manual_seed(rows + n)
    dt = DTYPES[dtype]
    x = torch.randn(rows, n, generator=g).to(dt)
    up = (torch.randn(experts, ff, n, generator=g) * n ** -0.5 * 1.5).to(dt)
    down = (torch.randn(experts, n, ff, generator=g) * ff ** -0.5).to(dt)
    ids = torch.stack([torch.randperm(experts, generator=g)[:top] for _ in range(rows)]).to(torch.int32)
    weights = torch.rand(rows, top, generator=g) * 0.8 + 0.1
    own = torch.randn(rows, n, generator=g).to(dt) if shared else None
    gate = torch.rand(rows, generator=g) if shared else None
    packed = ops.pack_experts(up.cuda(), down.cuda(), gated=False)
    assert (packed is not None) == (dtype == "bfloat16" and n % 8 == 0 and ff % 8 == 0)
    for on_input in (True, False):
        want = torch.zeros(rows, n, dtype=F64)
        for t in range(rows):
            for e, w in zip(ids[t].tolist(), weights[t].double()):
                a = plain_kunitar.squared_relu(up[e].double() @ ((w if on_input else 1.0) * x[t].double()))
                want[t] += (1.0 if on_input else w) * (down[e].double() @ a)
        if shared:
            want += gate.double()[:, None] * own.double()
        got = ops.apply_experts(x.cuda(), ids.cuda(), weights.cuda(), up.cuda(), down.cuda(), packed, own.cuda() if shared else None,
                                gate.cuda() if shared else None, activation="relu2", weight_on_input=on_input)
        _close(got, want, 5e-6 if dtype == "float32" else 1.5e-2, f"on input {on_input}")


# ------------------------------------------------- a window over cached latent vectors ---
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("heads, dim, rot, rank, vdim, page", [(4, 16, 16, 32, 24, 16), (8, 64, 16, 128, 80, 16), (3, 12, 6, 18, 10, 8), (20, 32, 32, 64, 32, 32)])
def test_one_key_at_every_edge_of_the_window(ops, dtype, heads, dim, rot, rank, vdim, page, monkeypatch):
    """A layer that reads vectors which another has cached: one key stands out and is placed just inside and just outside the
    window, at pages' borders and at the first position; rows decoded alone and in portions; one gate a head."""
    from tiny_llm_infer_amd.parts.base import GroupView, LayerCache
    g = torch.Generator().manual_seed(rank)
    dt, n = DTYPES[dtype], 90
    key = rank + rot
    pages = -(-n // page)
    order = torch.randperm(pages + 2, generator=g)
    tables = torch.full((1, pages + 1), -1, dtype=torch.int32)
    tables[0, :pages] = order[:pages]
    w_qk = (torch.randn(heads, rank, dim, generator=g) * dim ** -0.5).to(dt)
    w_v = (torch.randn(heads, vdim, rank, generator=g) * rank ** -0.5).to(dt)
    gates = torch.randn(n, heads + 3, generator=g).to(dt)
    query = torch.randn(n, heads * (dim + rot), generator=g).to(dt)
    cos, sin = torch.ones(n, rot // 2).cuda(), torch.zeros(n, rot // 2).cuda()          # (no turn: the scores are chosen below)
    scale = key ** -0.5
    q = query.double().view(n, heads, dim + rot)
    q_lat = torch.cat([torch.einsum("thd,hnd->thn", q[..., :dim], w_qk.double()), q[..., dim:]], dim=-1)
    for i, size in ((70, 1), (70, 2), (70, 33), (64, 16), (63, 48), (89, 33), (89, 90), (20, 40), (5, 6)):
        for back in {0, size - 1, size, i} & set(range(i + 1)):
            j = i - back
            keys = (torch.randn(n, key, generator=g) * 0.5)
            keys[j] = (q_lat[i].mean(dim=0) / q_lat[i].mean(dim=0).norm() * 40.0).float()       # the row at i looks for it
            keys = keys.to(dt)
            cached = torch.full((pages + 2, page, key), 30.0, dtype=dt)
            for t in range(n):
                cached[tables[0, t // page], t % page] = keys[t]
            kc = cached.cuda()
            group = GroupView(tensors={"latent": kc[None]}, tables=tables.cuda(), table_width=pages + 1, page_size=page, window=size)
            for first in (i, max(0, i - 13)):                                          # alone, and as the last row of a portion
                step = _view([first], [i + 1 - first], [0])
                rows = slice(first, i + 1)
                kd = keys.double()[:, None, :].expand(n, heads, key)
                want = plain_kunitar.windowed(q_lat[:i + 1], kd[:i + 1], kd[:i + 1, :, :rank], scale, size)[i]
                want = torch.einsum("hn,hen->he", want, w_v.double()) * torch.sigmoid(gates[i, 2:2 + heads].double())[:, None]
                for splits in ((None, 1, 3, 64) if first == i else (None,)):           # workgroups that share out a decoded row's keys
                    monkeypatch.setattr(ops, "sized_splits", splits)
                    got = ops.latent_attention(query[rows].cuda(), 0, None, step, LayerCache(group, 0, False), heads, dim, rot, rank, vdim,
                                               (cos, sin, rot), scale, w_qk.cuda(), w_v.cuda(), window=size, gate=(gates[rows].cuda(), 2))
                    _close(got[-1], want.reshape(-1), 1e-5 if dtype == "float32" else 2.5e-2,
                           f"row {i}, key {j}, window {size}, from {first}, {splits} splits")


@pytest.mark.parametrize("sinks", [False, True])
@pytest.mark.parametrize("window, keep", [(None, 0), (50, 0), (70, 20)])
def test_decoded_rows_whose_keys_are_shared_out(ops, sinks, window, keep, monkeypatch):
    """Rows of unequal length at once, all heads over one cached vector a position: any number of workgroups a row gives what one
    gives, kept first keys and sinks included."""
    from tiny_llm_infer_amd.parts.base import GroupView
    g = torch.Generator().manual_seed(4)
    lengths, page, heads, key, value = [1, 16, 17, 200, 333], 16, 20, 96, 64
    need = [-(-n // page) for n in lengths]
    ids, width, at = torch.randperm(sum(need), generator=g).to(torch.int32), max(need), 0
    tables = torch.full((len(lengths), width), -1, dtype=torch.int32)
    for i, n in enumerate(need):
        tables[i, :n] = ids[at:at + n]
        at += n
    kc = torch.randn(sum(need), 1, page, key, generator=g).to(torch.bfloat16).cuda()
    q = torch.randn(len(lengths), heads, key, generator=g).to(torch.bfloat16).cuda()
    group = GroupView(tensors={}, tables=tables.cuda(), table_width=width, page_size=page, window=window)
    step = _view([n - 1 for n in lengths], [1] * len(lengths), range(len(lengths)))
    extra = torch.randn(heads, generator=g).cuda() if sinks else None
    outs = []
    for splits in (1, 2, 5, 22, 64, None):
        monkeypatch.setattr(ops, "sized_splits", splits)
        outs.append(ops.sized_attention(q, step, group, kc, None, heads, 1, 1, key, value, 0.2, window, keep, torch.bfloat16, sinks=extra))
    monkeypatch.setattr(ops, "force_plain", True)
    plain = ops.sized_attention(q, step, group, kc, None, heads, 1, 1, key, value, 0.2, window, keep, torch.bfloat16, sinks=extra)
    for y in outs:
        _close(y, plain.cpu(), 2e-2, "against the plain kernel")
        _close(y, outs[0].cpu(), 1e-2, "against one workgroup")


# ------------------------------------------------------- one mixer alone, every cut ---
MIXERS = {
    "latent 4 x 16+8 -> 24": (L, _latent(4, 16, 8, 24, 32, 48, 20)),
    "latent 8 x 64+32 -> 64": (L, _latent(8, 64, 32, 64, 128, 96, 33)),
    "latent 20 x 32+16 -> 16": (L, _latent(20, 32, 16, 16, 48, 40, 65)),
    "latent 1 x 20+2 -> 7": (L, _latent(1, 20, 2, 7, 30, 9, 5, base=300.0)),
    "wkv 3 x 16": (W, _wkv(3, 16)),
    "wkv 2 x 20": (W, _wkv(2, 20)),
    "wkv 4 x 64": (W, _wkv(4, 64)),
    "wkv 2 x 128": (W, _wkv(2, 128)),
    "wkv 3 x 96": (W, _wkv(3, 96)),
}


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", list(MIXERS))
def test_one_mixer_alone_in_every_cut(tmp_path, name, dtype):
    """A model of one layer without feed-forward: the mixer between an embedding and the head."""
    kind, mixer = MIXERS[name]
    cfg = _config(120, 96, 8, [_layer(kind, mixer, None)])
    folder = write_folder(str(tmp_path / "one"), cfg, make_weights(cfg, 12, len(name), clear=dtype == "bfloat16"))
    reqs = _requests(120, [70, 45, 137, 33, 1, 58, 2, 3], seed=5)
    _all_cuts(folder, dtype, reqs, plain_logits(folder, reqs), 16, 384, TOL[dtype], name)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_a_state_that_remembers_a_token_hundreds_of_positions_back(tmp_path, dtype):
    """Channels that hardly decay: a token changed 400 positions back moves the last logits."""
    cfg = _config(90, 32, 8, [_layer(W, _wkv(2, 16), None), _layer(W, _wkv(1, 64), None)])
    w = make_weights(cfg, 8, 12, clear=dtype == "bfloat16")
    for i in range(2):
        w[f"l{i}.mix.w0"] = torch.full_like(w[f"l{i}.mix.w0"], -9.0)
    folder = write_folder(str(tmp_path / "long"), cfg, w)
    wd = plain_kunitar.read_model(folder)[1]
    toks = random_prompt(90, 430, 2)
    other = list(toks)
    other[30] = (toks[30] + 1) % 90
    want, moved = plain_kunitar.forward(cfg, wd, toks), plain_kunitar.forward(cfg, wd, other)
    assert np.abs(want[-1].numpy() - moved[-1].numpy()).max() > 50 * TOL["float32"] * np.abs(want[-1].numpy()).max()
    reqs = {"r0": toks, "r1": other, "r2": toks[:77]}
    full = {"r0": want.numpy(), "r1": moved.numpy(), "r2": want.numpy()[:77]}
    for steps in (trace_whole(reqs), trace_prefill_then_decode(reqs, tail=40), trace_portions(reqs, seed=5), trace_mixed(reqs, max_tokens=1024, seed=2)):
        got = collect(steps, _replay(_runner(folder, dtype, 1024, 16), steps))
        for rid in reqs:
            err, row, scale = max_error(got[rid], full[rid])
            assert err <= 2 * TOL[dtype] * scale, (rid, err, row)


# ------------------------------------------------------------- the model, every cut ---
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", list(SMALL))
def test_all_cuts_match_plain(folders, clear_folders, name, dtype):
    folder = (clear_folders if dtype == "bfloat16" else folders)[name]
    reqs = _requests(SMALL[name][0]["vocab"], [70, 45, 197, 33, 1, 58, 2, 3], seed=5)
    _all_cuts(folder, dtype, reqs, plain_logits(folder, reqs), SMALL[name][2], 384, TOL[dtype], name)


def test_token_by_token_from_the_first(folders):
    for name in ("A", "B"):
        folder = folders[name]
        reqs = _requests(SMALL[name][0]["vocab"], [60], seed=21)
        want = plain_logits(folder, reqs)
        steps = trace_prefill_then_decode(reqs, tail=59)
        got = collect(steps, _replay(_runner(folder, "float32", 64, SMALL[name][2]), steps))
        err, row, scale = max_error(got["r0"], want["r0"])
        assert err <= TOL["float32"] * scale, (name, err, row)


def test_unequal_requests_together_equal_each_alone(folders):
    folder = folders["R"]
    reqs = _requests(320, [3, 130, 34, 65], seed=60)
    alone = {rid: _replay(_runner(folder, "float32", 256, 32), trace_whole({rid: toks}))[0] for rid, toks in reqs.items()}
    step = {"step": 0, "entries": [{"id": r, "tokens": t, "want": list(range(len(t)))} for r, t in reqs.items()], "end": list(reqs)}
    together = collect([step], _replay(_runner(folder, "float32", 512, 32), [step]))
    for rid in reqs:
        assert np.abs(together[rid] - alone[rid]).max() <= 2e-5 * np.abs(alone[rid]).max()


def test_bfloat16_through_the_plain_kernels(clear_folders):
    """The plain twins of all tuned kernels, bfloat16, in every cut."""
    from tiny_llm_infer_amd.engine.loading import load_model
    from tiny_llm_infer_amd.engine.runner import ModelRunner
    from tiny_llm_infer_amd.kernels.ops import HipOps
    for name in ("A", "R"):
        folder, page = clear_folders[name], SMALL[name][2]
        reqs = _requests(SMALL[name][0]["vocab"], [70, 45, 97, 33, 1, 58], seed=15)
        want = plain_logits(folder, reqs)
        for steps in (trace_whole(reqs), trace_portions(reqs, seed=3), trace_mixed(reqs, max_tokens=256, seed=9)):
            ops = HipOps("cuda:0")
            ops.use_plain_kernels()
            model, _ = load_model(folder, "bfloat16", "cuda:0", max_model_len=512, ops=ops)
            runner = ModelRunner(model, model.env, page_size=page, num_pages=256 // page, max_requests=4, max_batch_tokens=512)
            got = collect(steps, _replay(runner, steps))
            for rid in reqs:
                err, row, scale = max_error(got[rid], want[rid])
                assert err <= TOL["bfloat16"] * scale, (name, rid, err, row)


def test_long_decoding_through_recorded_launches(clear_folders):
    """150 tokens decoded one by one for three requests at once (bfloat16: the steps are replayed from recordings): the
    windows pass over decoded tokens, pages are given back."""
    folder = clear_folders["R"]
    reqs = _requests(320, [160, 171, 183], seed=77)
    want = plain_logits(folder, reqs)
    runner = _runner(folder, "bfloat16", 768, 32)
    steps = [{"step": 0, "entries": [{"id": r, "tokens": t[:len(t) - 150], "want": []} for r, t in reqs.items()], "end": []}]
    for j in range(150):
        steps.append({"step": j + 1, "entries": [{"id": r, "tokens": [t[len(t) - 150 + j]], "want": [0]} for r, t in reqs.items()],
                      "end": list(reqs) if j == 149 else []})
    got = collect(steps, _replay(runner, steps))
    assert runner.graph_replays > 100
    for rid, toks in reqs.items():
        err, row, scale = max_error(got[rid], want[rid][len(toks) - 150:])
        assert err <= TOL["bfloat16"] * scale, (rid, err, row)


def test_recorded_steps_equal_eager_steps(clear_folders):
    """The same decode steps replayed from recordings and run eagerly, many rows (products of every size class), with the
    program's own work between the replays."""
    from tiny_llm_infer_amd.engine.replay import Replayer
    folder = clear_folders["R"]
    reqs = _requests(320, [20 + i % 7 for i in range(40)], seed=9)
    outs = []
    for graphs in (True, False):
        runner = _runner(folder, "bfloat16", 40 * 64, 32, max_requests=40)
        runner.use_graphs = runner.use_graphs and graphs
        steps = [{"step": 0, "entries": [{"id": r, "tokens": t[:10], "want": []} for r, t in reqs.items()], "end": []}]
        for j in range(10, 20):
            steps.append({"step": len(steps), "entries": [{"id": r, "tokens": [t[j]], "want": [0]} for r, t in reqs.items()], "end": []})
        got, rp = [], Replayer(runner)
        for st in steps:
            got.append(rp.run_step(st))
            torch.cuda.synchronize()
            torch.randn(1000, device="cuda").sum()
        assert (runner.graph_replays > 0) == graphs
        outs.append(got[1:])
    for a, b in zip(*outs):
        assert np.abs(a - b).max() <= 2e-2 * np.abs(b).max()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_greedy_generation_through_the_engine(folders, clear_folders, dtype):
    from tiny_llm_infer_amd.engine.llm_engine import LLMEngine
    from tiny_llm_infer_amd.sampling.params import SamplingParams
    folder = (clear_folders if dtype == "bfloat16" else folders)["A"]
    prompts = [random_prompt(160, n, 90 + n) for n in (4, 19, 30, 41)]
    eng = LLMEngine.from_folder(folder, dtype=dtype, max_model_len=128, page_size=16, num_kv_blocks=32, max_num_seqs=3,
                                max_num_batched_tokens=32)
    got = eng.generate(prompts, SamplingParams(max_tokens=10, ignore_eos=True))
    if dtype == "float32":
        assert [r.token_ids for r in got] == [plain_greedy(folder, p, 10) for p in prompts]
    else:
        # rounding may turn a close call: every token must be the plain implementation's choice or within
        # the rounding error of it, given the tokens before
        cfg, w = plain_kunitar.read_model(folder)
        for p, r in zip(prompts, got):
            logits = plain_kunitar.forward(cfg, w, p + r.token_ids)[len(p) - 1:-1]
            for z, t in zip(logits, r.token_ids):
                assert float(z.max() - z[t]) <= 2 * TOL["bfloat16"] * float(z.abs().max())
    eng.runner.cache.check()
    assert eng.runner.cache.free_pages() == eng.runner.cache.pages_per_group()


# ------------------------------------------------------------------ the command line ---
def test_the_programs_take_a_kunitar_folder(folders, tmp_path):
    """bin/trace_run replays a mixed trace, model_main --infer generates greedily, and a model of random
    weights made from a config.json alone loads and generates."""
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    folder, vocab = folders["B"], SMALL["B"][0]["vocab"]
    reqs = _requests(vocab, [40, 9, 77, 23, 52], seed=12)
    want = plain_logits(folder, reqs)
    steps = trace_mixed(reqs, max_tokens=192, seed=4)
    proc = subprocess.run([sys.executable, os.path.join(root, "bin", "trace_run"), "--model", folder, "--dtype", "float32",
                           "--out", str(tmp_path / "out"), "--max-tokens", "192"],
                          input="".join(json.dumps(s) + "\n" for s in steps), text=True, stdout=subprocess.PIPE,
                          stderr=subprocess.PIPE, timeout=600)
    assert proc.returncode == 0, proc.stderr[-2000:]
    assert proc.stdout.split("\n")[:-1] == [f"done {s['step']}" for s in steps]
    outputs = {s["step"]: np.fromfile(tmp_path / "out" / f"{s['step']}.f32", dtype="<f4").reshape(-1, vocab)
               for s in steps if sum(len(e["want"]) for e in s["entries"])}
    got = collect(steps, outputs)
    for rid in reqs:
        err, row, scale = max_error(got[rid], want[rid])
        assert err <= TOL["float32"] * scale, (rid, err, row)
    prompt = random_prompt(vocab, 21, 3)
    proc = subprocess.run([sys.executable, os.path.join(root, "bin", "model_main"), "--infer", "--model", folder, "--dtype",
                           "float32", "--prompt-ids", ",".join(map(str, prompt)), "--max-new-tokens", "8", "--ignore-eos",
                           "--max-seq-len", "64", "--num-kv-blocks", "16"],
                          text=True, stdout=subprocess.PIPE, stderr=subprocess.PIPE, timeout=600)
    assert proc.returncode == 0, proc.stderr[-2000:]
    assert [int(t) for t in proc.stdout.split()] == plain_greedy(folder, prompt, 8)
    cfg_file = tmp_path / "config.json"
    cfg_file.write_text(json.dumps(SMALL["R"][0]))
    proc = subprocess.run([sys.executable, os.path.join(root, "bin", "model_main"), "--infer", "--config", str(cfg_file),
                           "--random-weights", "--seed", "5", "--prompt-ids", "1,2,3,4,5", "--max-new-tokens", "6",
                           "--ignore-eos", "--max-seq-len", "64", "--num-kv-blocks", "16"],
                          text=True, stdout=subprocess.PIPE, stderr=subprocess.PIPE, timeout=600)
    assert proc.returncode == 0, proc.stderr[-2000:]
    assert len(proc.stdout.split()) == 6
