"""Kosusun on the GPU: each mechanism's kernels alone against the plain implementation's function for
it (keys just inside and outside the window, blocks just seen and not yet, keys far back), then the
model through the step function in every cut, in float32 and in bfloat16, long decoding through
recorded launches, and greedy generation through the engine and the command line."""
import json
import math
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

import plain_kosusun
from helpers import collect, max_error, random_prompt, trace_mixed, trace_portions, trace_prefill_then_decode, trace_whole
from kosusun_helpers import (SMALL, _config, _layer, _mlstm, _parallel, _retention, _rot, _window, make_weights, plain_greedy,
                             plain_logits, write_folder)

pytestmark = pytest.mark.gpu
F64 = torch.float64
# of the largest logit
TOL = {"float32": 2e-5, "bfloat16": 4e-2}
DTYPES = {"float32": torch.float32, "bfloat16": torch.bfloat16}


@pytest.fixture(scope="module")
def ops():
    from tiny_llm_infer_amd.kernels.ops import HipOps
    return HipOps("cuda:0")


@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    root = tmp_path_factory.mktemp("kosusun")
    return {name: write_folder(str(root / name), cfg, make_weights(cfg, seed)) for name, (cfg, _, seed) in SMALL.items()}


@pytest.fixture(scope="module")
def mild_folders(tmp_path_factory):
    """Weights whose attention scores are smaller (for bfloat16)."""
    root = tmp_path_factory.mktemp("kosusun_mild")
    return {name: write_folder(str(root / name), cfg, make_weights(cfg, seed, mild=True)) for name, (cfg, _, seed) in SMALL.items()}


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


# ------------------------------------------------- the window, the blocks and the sink, alone ---
class _Pages:
    """Pages for tokens and for blocks of a few sequences, dealt out in a shuffled order, with what others left in them."""

    def __init__(self, lengths, kv_heads, dim, vdim, pool, page, dtype, seed):
        from tiny_llm_infer_amd.parts.base import GroupView, LayerCache
        rng = np.random.default_rng(seed)

        def group(span, stride):
            need = [-(-n // span) for n in lengths]
            ids = rng.permutation(sum(need) + 3)
            width, tables, at = max(need) + 1, [], 0
            for n in need:
                tables.append(list(ids[at:at + n]) + [-1] * (width - n))
                at += n
            pages = sum(need) + 3
            return GroupView(tensors={"k": torch.full((1, pages, kv_heads, page, dim), 2.0, dtype=dtype, device="cuda"),
                                      "v": torch.full((1, pages, kv_heads, vdim, page), -9.0, dtype=dtype, device="cuda")},
                             tables=torch.tensor(np.array(tables), dtype=torch.int32, device="cuda"), table_width=width,
                             page_size=page, window=None, stride=stride)
        self.tokens, self.blocks = group(page, 1), group(page * pool, pool)
        self.LayerCache = LayerCache

    def cache(self, live):
        import dataclasses
        pick = lambda g: dataclasses.replace(g, tables=g.tables[live].contiguous())
        return self.LayerCache(pick(self.tokens), 0, True, [self.LayerCache(pick(self.blocks), 0, True)])


def _attend(ops, q, k, v, scale, window, pool, sinks, page, cuts, out_scale=1.0, seed=0):
    """The attention op over sequences given as q, k, v [T, heads, size], in portions of ``cuts`` rows: its outputs."""
    dtype = q[0].dtype
    H, d, G, e = q[0].shape[1], q[0].shape[2], k[0].shape[1], v[0].shape[2]
    lengths = [len(x) for x in q]
    pages = _Pages(lengths, G, d, e, pool, page, dtype, seed)
    proj = [torch.cat([torch.zeros(n, 8, dtype=dtype)] + [t[i].reshape(n, -1) for t in (q, k, v)], dim=1) for i, n in enumerate(lengths)]
    out_width = (H * e + 16 + 7) // 8 * 8
    got = [[] for _ in lengths]
    for starts, counts, live in _portions(lengths, cuts):
        rows = torch.cat([proj[i][s:s + c] for i, s, c in zip(live, starts, counts)]).contiguous().cuda()
        out = torch.full((len(rows), out_width), 5.0, dtype=dtype, device="cuda")
        ops.pooled_window_attention(rows, 8, _view(starts, counts, live), pages.cache(live), H, G, d, e, None, None, None, 0.0, None,
                                    scale, None if sinks is None else sinks.cuda(), window, pool, out, 8, out_scale)
        assert (out[:, :8] == 5.0).all() and (out[:, 8 + H * e:] == 5.0).all()          # its columns and no others
        r = 0
        for i, c in zip(live, counts):
            got[i].append(out[r:r + c, 8:8 + H * e].reshape(c, H, e).cpu())
            r += c
    return [torch.cat(g) for g in got]


SIZES = [  # heads, kv heads, key size, value size, window, pool, page
    (4, 2, 16, 32, 20, 4, 16), (6, 2, 64, 64, 33, 12, 16), (4, 1, 128, 128, 40, 16, 32), (3, 3, 20, 12, 7, 10, 8),
    (2, 1, 48, 80, 16, 1, 16), (6, 3, 64, 64, 20, 6, 8), (3, 1, 128, 128, 70, 2, 64), (8, 1, 64, 64, 1, 1, 16), (34, 2, 16, 16, 1, 3, 16), (2, 2, 256, 144, 25, 5, 64), (1, 1, 7, 5, 30, 8, 4), (18, 1, 288, 64, 50, 7, 16),
]


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("sizes", SIZES, ids=lambda s: "-".join(map(str, s)))
@pytest.mark.parametrize("own", [True, False], ids=["own", "sized"])
def test_window_and_blocks_in_portions(ops, dtype, sizes, own, monkeypatch):
    """Sequences of unequal lengths side by side, in portions of 1 to 70 rows and row by row."""
    H, G, d, e, window, pool, page = sizes
    if not own and (dtype == "float32" or not ops.lib.tli_pooled_prefill_takes(d, e, page, 200, window, pool)):
        pytest.skip("no prefill kernel of their own")
    monkeypatch.setattr(ops, "pooled_prefill", own)
    g = torch.Generator().manual_seed(d + e)
    lengths = [150, 1, 67, pool + window]
    dt = DTYPES[dtype]
    make = lambda n, h, s, std: (torch.randn(n, h, s, generator=g) * std).to(dt)
    q = [make(n, H, d, 1.5) for n in lengths]
    k, v = [make(n, G, d, 1.0) for n in lengths], [make(n, G, e, 1.0) for n in lengths]
    sinks = torch.randn(H, generator=g) + 1.0
    want = [plain_kosusun.windowed_attention(a.double(), b.double(), c.double(), d ** -0.5, window, pool, sinks) for a, b, c in zip(q, k, v)]
    for cuts in ([1000], [1, 43, 2, 16, 70, 7], [1]):
        got = _attend(ops, q, k, v, d ** -0.5, window, pool, sinks, page, cuts, out_scale=0.5)
        for i, n in enumerate(lengths):
            _close(got[i], 0.5 * want[i], 1e-5 if dtype == "float32" else 2e-2, f"sequence {i} in portions of {cuts}")
    if dtype == "bfloat16" and ops.lib.tli_attention_sized_mfma_takes(d, e, page, 1):
        for splits in (2, 5, 64):                       # a row's keys shared out over workgroups, some of which have none
            monkeypatch.setattr(ops, "pooled_splits", splits)
            got = _attend(ops, q, k, v, d ** -0.5, window, pool, sinks, page, [1], out_scale=0.5)
            for i, n in enumerate(lengths):
                _close(got[i], 0.5 * want[i], 2e-2, f"sequence {i} row by row in {splits} splits")
        monkeypatch.setattr(ops, "pooled_splits", None)
    got = _attend(ops, q, k, v, d ** -0.5, window, pool, None, page, [29, 64])
    for i in range(len(lengths)):
        bare = plain_kosusun.windowed_attention(q[i].double(), k[i].double(), v[i].double(), d ** -0.5, window, pool, None)
        _close(got[i], bare, 1e-5 if dtype == "float32" else 2e-2, f"sequence {i} without a sink")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("sizes", [(4, 2, 16, 32, 20, 4, 16), (4, 2, 64, 64, 37, 12, 16), (2, 1, 128, 128, 40, 16, 32), (2, 1, 20, 12, 7, 10, 8)],
                         ids=lambda s: "-".join(map(str, s)))
def test_one_key_at_every_edge(ops, dtype, sizes, monkeypatch):
    """One key answers the last row's query far above all others.  It stands just inside and just outside the window
    (there in no block that is seen, or in the last one that is), in the first and last position of blocks, at the
    borders of pages, at position 0 and hundreds back; in a prompt, at the end of a portion of two, and decoded alone.
    The same with a window one longer or shorter, or blocks that come one position early or late, would give
    something else wherever the edge is what matters (checked on the plain implementation)."""
    H, G, d, e, window, pool, page = sizes
    g = torch.Generator().manual_seed(window)
    dt = DTYPES[dtype]
    told = 0
    for n in (350, 350 - 350 % pool + window, 349 - 350 % pool + window):          # the last row ends no block, and just sees one or not yet
        i = n - 1
        edge = i - window + 1                                                      # first position inside the window
        seen = max(0, edge // pool)                                                # blocks that are seen
        places = {0, 1, pool - 1, pool, page - 1, page, edge, edge - 1, edge + 1, seen * pool, seen * pool - 1, (seen - 1) * pool,
                  seen * pool + 1, i, i - 1, 17 * pool}
        q = (torch.randn(n, H, d, generator=g) * 0.1).to(dt)
        k = (torch.randn(n, G, d, generator=g) * 0.1).to(dt)
        v = torch.randn(n, G, e, generator=g).to(dt)
        u = torch.randn(d, generator=g)
        u = u / u.norm()
        q[i] = (u * 8.0).to(dt)
        for at in sorted(p for p in places if 0 <= p <= i):
            kk = k.clone()
            kk[at] = (u * 2.0 * pool).to(dt)                                       # (as one of a block's mean still a score of 16)
            want = _last_row(q, kk, v, window, pool)
            for other in (window - 1, window + 1):
                told += float((_last_row(q, kk, v, other, pool) - want).abs().max()) > 0.1 * float(want.abs().max())
            for cuts, splits in (([n], None), ([n - 2, 2], None), ([n - 1, 1], None), ([n - 1, 1], 3)):
                monkeypatch.setattr(ops, "pooled_splits", splits)
                got = _attend(ops, [q], [kk], [v], 1.0, window, pool, None, page, cuts)[0][i]
                _close(got, want, 1e-5 if dtype == "float32" else 2e-2, f"{n} rows in {cuts}, the key at {at} (window from {edge}, {seen} blocks)")
    assert told >= 4


def _last_row(q, k, v, window, pool):
    """The last row's outputs [H, e], the window and blocks by the plain implementation's rules."""
    q, k, v = q.double(), k.double(), v.double()
    i, H, G = len(q) - 1, q.shape[1], k.shape[1]
    t, b = plain_kosusun.seen_tokens(i, window), plain_kosusun.seen_blocks(i, window, pool)
    keys = torch.cat([k[t], plain_kosusun.pooled_blocks(k, pool)[b]]) if b else k[t]
    values = torch.cat([v[t], plain_kosusun.pooled_blocks(v, pool)[b]]) if b else v[t]
    return torch.stack([plain_kosusun.softmax_with_sink(keys[:, h // (H // G)] @ q[i, h], None) @ values[:, h // (H // G)] for h in range(H)])


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_blocks_of_more_sequences_than_a_wave_has_lanes(ops, dtype):
    g = torch.Generator().manual_seed(8)
    lengths = [1 + (7 * i) % 23 for i in range(150)]
    q, k, v = ([torch.randn(n, h, 16, generator=g).to(DTYPES[dtype]) for n in lengths] for h in (2, 1, 1))
    for cuts in ([30], [3, 9, 2]):
        got = _attend(ops, q, k, v, 0.25, 5, 3, None, 16, cuts)
        for i in range(len(lengths)):
            want = plain_kosusun.windowed_attention(q[i].double(), k[i].double(), v[i].double(), 0.25, 5, 3, None)
            _close(got[i], want, 1e-5 if dtype == "float32" else 2e-2, f"sequence {i} in portions of {cuts}")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_a_sink_that_takes_most_of_the_weight(ops, dtype, monkeypatch):
    g = torch.Generator().manual_seed(5)
    dt = DTYPES[dtype]
    q, k, v = ((torch.randn(90, h, 16, generator=g)).to(dt) for h in (3, 1, 1))
    for sinks in (torch.tensor([9.0, -30.0, 2.0]), torch.tensor([80.0, 5.0, 0.0])):
        want = plain_kosusun.windowed_attention(q.double(), k.double(), v.double(), 0.25, 24, 6, sinks)
        for cuts, splits in (([90], None), ([30, 1], None), ([30, 1], 4)):
            monkeypatch.setattr(ops, "pooled_splits", splits)
            _close(_attend(ops, [q], [k], [v], 0.25, 24, 6, sinks, 16, cuts)[0], want, 1e-5 if dtype == "float32" else 2e-2, f"{sinks} {cuts}")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("heads, kv_heads, dim, vdim, dims, factor, pairing", [
    (4, 2, 16, 24, 8, 4.0, "interleaved"), (3, 1, 20, 12, 20, 1.0, "interleaved"), (2, 2, 64, 64, 32, 2.0, "half"), (5, 5, 7, 3, 2, 1.0, "interleaved")])
def test_norms_over_the_projection_rotation_and_bias(ops, dtype, heads, kv_heads, dim, vdim, dims, factor, pairing):
    """What stands before the attention: seen through a window that holds everything and scores that matter."""
    from tiny_llm_infer_amd.parts.base import BuildEnv, build_part
    from tiny_llm_infer_amd.config.base import PartSpec
    g = torch.Generator().manual_seed(dim)
    dt, n, eps, base = DTYPES[dtype], 61, 1e-2, 100.0
    sizes = (heads * dim, kv_heads * dim, kv_heads * vdim)
    proj = torch.randn(n, sum(sizes), generator=g).to(dt)
    bias = torch.randn(sum(sizes), generator=g) * 0.5
    qw, kw = torch.randn(sizes[0], generator=g) * 0.3 + 1.0, torch.randn(sizes[1], generator=g) * 0.3 + 1.0
    x = proj.double() + bias.double()
    rot = {"dims": dims, "base": base, "scaling": {"factor": factor}}
    pos, near = torch.arange(n), pairing == "interleaved"
    q = plain_kosusun.turn(plain_kosusun.weighted_norm(x[:, :sizes[0]], qw.double(), eps).view(n, heads, dim), pos, rot, near)
    k = plain_kosusun.turn(plain_kosusun.weighted_norm(x[:, sizes[0]:sizes[0] + sizes[1]], kw.double(), eps).view(n, kv_heads, dim), pos, rot, near)
    v = x[:, sizes[0] + sizes[1]:].view(n, kv_heads, vdim)
    want = plain_kosusun.windowed_attention(q, k, v, 0.3, 100, 5, None)
    part = build_part("position", PartSpec("rope_interleaved" if near else "rope_neox", {
        "head_dim": dim, "rotary_dim": dims, "theta": base, "max_positions": 128, "scaling_factor": factor, "angles": "float64"}))
    part.load({}, BuildEnv(dtype=dt, device=torch.device("cuda:0"), ops=ops, max_model_len=128))
    pages = _Pages([n], kv_heads, dim, vdim, 5, 16, dt, 1)
    got = []
    for starts, counts, live in _portions([n], [20, 1, 30]):
        out = torch.zeros((counts[0], (heads * vdim + 7) // 8 * 8), dtype=dt, device="cuda")
        ops.pooled_window_attention(proj[starts[0]:starts[0] + counts[0]].contiguous().cuda(), 0, _view(starts, counts, live), pages.cache(live), heads, kv_heads,
                                    dim, vdim, bias.cuda(), qw.cuda(), kw.cuda(), eps, part.rotary(), 0.3, None, 100, 5, out, 0, 1.0)
        got.append(out[:, :heads * vdim].reshape(counts[0], heads, vdim).cpu())
    _close(torch.cat(got), want, 1e-5 if dtype == "float32" else 2e-2, "prepared rows")


# --------------------------------------------------------------- the recurrences, alone ---
RECURRENT = [(2, 16, 24), (3, 20, 12), (1, 40, 20), (4, 64, 32), (2, 128, 128), (1, 200, 50), (5, 8, 7), (1, 256, 16), (2, 64, 64), (3, 48, 112), (2, 96, 16)]


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("lengths, cuts", [([61, 97, 45], [1, 43, 2, 16, 33, 7]), ([900, 30, 301], [700, 390, 1, 2]), ([24, 20, 3], [1])])
@pytest.mark.parametrize("heads, dk, dv", RECURRENT)
@pytest.mark.parametrize("chunks", [True, False], ids=["chunks", "rows"])
def test_retention_in_portions_and_slots_that_are_used_again(ops, dtype, heads, dk, dv, lengths, cuts, chunks, monkeypatch):
    """Sequences side by side in portions down to one row, also long ones that are walked in segments; then
    others in the same slots, which are never cleared."""
    from tiny_llm_infer_amd.parts.base import BuildEnv, build_part
    from tiny_llm_infer_amd.config.base import PartSpec
    if chunks and (dtype == "float32" or dk % 16 or dv % 16 or max(dk, dv) > 128):
        pytest.skip("these rows do not go through chunks")
    monkeypatch.setattr(ops, "recurrence_in_chunks", chunks)
    if max(lengths) > 500 and (dk > 128 or heads > 2):
        lengths = [min(n, 480) for n in lengths]
    g = torch.Generator().manual_seed(dk * dv)
    dt = DTYPES[dtype]
    decay = torch.linspace(0.8, 1.0, heads)
    dims = max(2, dk // 2 // 2 * 2)
    m = {"heads": heads, "dim": dk, "vdim": dv, "decay": decay.tolist(), "rot": {"dims": dims, "base": 1000.0}}
    width = 2 * heads * dk + 2 * heads * dv
    eye = torch.eye(width, dtype=F64)
    names = {"q": eye[:heads * dk], "k": eye[heads * dk:2 * heads * dk], "v": eye[2 * heads * dk:2 * heads * dk + heads * dv],
             "g": eye[2 * heads * dk + heads * dv:], "o": torch.eye(heads * dv, dtype=F64)}
    part = build_part("position", PartSpec("rope_neox", {"head_dim": dk, "rotary_dim": dims, "theta": 1000.0, "max_positions": 1024,
                                                         "angles": "float64"}))
    part.load({}, BuildEnv(dtype=dt, device=torch.device("cuda:0"), ops=ops, max_model_len=1024))
    state = torch.full((3, *ops.lightning_state_shape(heads, dk, dv)), 7.0, device="cuda")       # what another request left
    for slots in ([0, 1, 2], [2, 0, 1]):
        proj = [(torch.randn(n, width, generator=g)).to(dt) for n in lengths]
        for p in proj:
            p[:, heads * dk:2 * heads * dk] += p[:, :heads * dk]                                 # (no output that is all rounding)
        got = [[] for _ in lengths]
        for starts, counts, live in _portions(lengths, cuts):
            pad = 8 if chunks else 3
            rows = torch.cat([torch.zeros(sum(counts), pad, dtype=dt), torch.cat([proj[i][s:s + c] for i, s, c in zip(live, starts, counts)])], dim=1).cuda()
            y = torch.full((len(rows), (heads * dv + 15) // 8 * 8), 4.0, dtype=dt, device="cuda")
            ops.retention(rows, pad, decay.cuda(), state, _view(starts, counts, [slots[i] for i in live]), heads, dk, dv, part.rotary(), dk ** -0.5,
                          1e-5, 0.7, y, 8)
            assert (y[:, :8] == 4.0).all() and (y[:, 8 + heads * dv:] == 4.0).all()
            r = 0
            for i, c in zip(live, counts):
                got[i].append(y[r:r + c, 8:8 + heads * dv].cpu())
                r += c
        for i in range(len(lengths)):
            want = 0.7 * plain_kosusun.retention(proj[i].double(), m, names, "", 1e-5)
            _close(torch.cat(got[i]), want, 5e-5 if dtype == "float32" else 1.5e-2, f"sequence {i} in slot {slots[i]}")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("lengths, cuts", [([61, 97, 45], [1, 43, 2, 16, 33, 7]), ([900, 30, 301], [700, 390, 1, 2]), ([24, 20, 3], [1])])
@pytest.mark.parametrize("heads, dk, dv", RECURRENT)
@pytest.mark.parametrize("chunks", [True, False], ids=["chunks", "rows"])
def test_matrix_memory_in_portions_and_slots_that_are_used_again(ops, dtype, heads, dk, dv, lengths, cuts, chunks, monkeypatch):
    """As the retention's test; gates that open and close, so that the running maximum is taken over again and again, and
    a head whose forget gate is open throughout."""
    if chunks and (dtype == "float32" or dk % 16 or dv % 16 or max(dk, dv) > 128):
        pytest.skip("these rows do not go through chunks")
    monkeypatch.setattr(ops, "recurrence_in_chunks", chunks)
    if max(lengths) > 500 and (dk > 128 or heads > 2):
        lengths = [min(n, 480) for n in lengths]
    g = torch.Generator().manual_seed(dk + dv)
    dt, cap = DTYPES[dtype], 6.0
    m = {"heads": heads, "dim": dk, "vdim": dv, "gate_cap": cap}
    wide = 2 * heads * dk + 2 * heads * dv
    eye = torch.eye(wide + 2 * heads, dtype=F64)
    n = 4 * heads + (8 if dk % 8 == 0 else 3)                        # the layer's input, which only the gates read here
    w_gates = (torch.randn(2 * heads, n, generator=g) * 2 * n ** -0.5).to(dt)
    bias = torch.randn(2 * heads, generator=g)
    bias[heads:] += 3.0
    bias[heads] = 40.0
    at = [0, heads * dk, 2 * heads * dk, 2 * heads * dk + heads * dv, wide, wide + heads, wide + 2 * heads]
    names = {r: eye[a:b] for r, a, b in zip(("q", "k", "v", "g", "i", "f"), at, at[1:])}
    weight = torch.randn(heads * dv, generator=g) * 0.2 + 1.0
    names.update({"o": torch.eye(heads * dv, dtype=F64), "norm": weight.double(), "i.b": bias[:heads].double(), "f.b": bias[heads:].double()})
    state = torch.full((3, *ops.mlstm_state_shape(heads, dk, dv)), 7.0, device="cuda")
    maxima = torch.full((3, heads), 50.0, device="cuda")
    for slots in ([0, 1, 2], [2, 0, 1]):
        proj = [(torch.randn(n, wide, generator=g)).to(dt) for n in lengths]
        x = [torch.randn(c, n, generator=g).to(dt) for c in lengths]
        for p in proj:
            p[:, heads * dk:2 * heads * dk] += p[:, :heads * dk]
        got = [[] for _ in lengths]
        for k, (starts, counts, live) in enumerate(_portions(lengths, cuts + [1])):
            pad = 8 if chunks else 5
            rows = torch.cat([torch.zeros(sum(counts), pad, dtype=dt), torch.cat([proj[i][s:s + c] for i, s, c in zip(live, starts, counts)])], dim=1).cuda()
            inputs = torch.cat([x[i][s:s + c] for i, s, c in zip(live, starts, counts)]).cuda()
            if k % 3 == 2 and dtype == "bfloat16":                                               # rows that still owe a factor of 1/2, in three parts
                from tiny_llm_infer_amd.kernels.ops import NormedRows
                inputs = NormedRows((inputs.float() * 2).to(dt), torch.full((3, len(rows)), n * 3.9 / 3, device="cuda"), 0.1)
            y = torch.full((len(rows), (heads * dv + 7) // 8 * 8), 4.0, dtype=dt, device="cuda")
            ops.mlstm(rows, pad, inputs, w_gates.cuda(), bias.cuda(), cap, state, maxima, _view(starts, counts, [slots[i] for i in live]), heads, dk, dv,
                      dk ** -0.5, weight.cuda(), 1e-5, 1.3, y, 0)
            assert (y[:, heads * dv:] == 4.0).all()
            r = 0
            for i, c in zip(live, counts):
                got[i].append(y[r:r + c, :heads * dv].cpu())
                r += c
        for i in range(len(lengths)):
            want = 1.3 * plain_kosusun.mlstm(torch.cat([proj[i].double(), x[i].double() @ w_gates.double().T], dim=1), m, names, "", 1e-5)
            _close(torch.cat(got[i]), want, 5e-5 if dtype == "float32" else 1.5e-2, f"sequence {i} in slot {slots[i]}")


# ------------------------------------------------------- the gated products' activation ---
@pytest.mark.parametrize("rows", [1, 16, 33, 100, 200, 700])
@pytest.mark.parametrize("n, inter", [(128, 96), (256, 512), (72, 40), (100, 37)])
def test_gated_product_with_gelu_in_shared_rows(ops, rows, n, inter):
    """act(gate) * up * scale for both activations into columns of a wider buffer, through every product kernel."""
    from tiny_llm_infer_amd.parts.base import BuildEnv
    from tiny_llm_infer_amd.parts.linear import GatedMatrix
    g = torch.Generator().manual_seed(rows + n)
    for dt, tol in ((torch.bfloat16, 1e-2), (torch.float32, 2e-6)):
        env = BuildEnv(dtype=dt, device=torch.device("cuda:0"), ops=ops, max_model_len=128)
        x = torch.randn(rows, n, generator=g).to(dt)
        gate, up = ((torch.randn(inter, n, generator=g) * n ** -0.5 * 2).to(dt) for _ in range(2))
        m = GatedMatrix(gate.cuda(), up.cuda(), env)
        a, b = x.double() @ gate.double().T, x.double() @ up.double().T
        for act, want in (("gelu_tanh", plain_kosusun.gelu_tanh(a) * b), ("silu", a * torch.sigmoid(a) * b)):
            out = torch.full((rows, 16 + (inter + 7) // 8 * 8 + 8), 3.0, dtype=dt, device="cuda")
            ops.linear_swiglu(x.cuda(), m, activation=act, scale=0.3, into=(out, 16))
            _close(out[:, 16:16 + inter], 0.3 * want, tol, f"{act} {dt}")
            assert (out[:, :16] == 3.0).all() and (out[:, 16 + inter:] == 3.0).all()
            _close(ops.linear_swiglu(x.cuda(), m, activation=act), want, tol, f"{act} {dt} alone")


# ------------------------------------------------------- one mixer alone, every cut ---
_R = _retention(2, 16, 16, [0.9, 0.98], _rot(8))
MIXERS = {
    "window 4/2 16 -> 24": ("parallel", _parallel(_window(4, 2, 16, 24, 20, 4, _rot(8, factor=4.0)), _R)),
    "window 8/2 64 -> 64": ("parallel", _parallel(_window(8, 2, 64, 64, 48, 16, _rot(64)), _R)),
    "window 4/4 128 -> 128": ("parallel", _parallel(_window(4, 4, 128, 128, 33, 6, _rot(64, factor=2.0)), _R, 0.4, 0.2)),
    "window 5/1 20 -> 12": ("parallel", _parallel(_window(5, 1, 20, 12, 9, 11, _rot(2)), _R)),
    "window 20/1 32 -> 16": ("parallel", _parallel(_window(20, 1, 32, 16, 24, 3, _rot(32)), _R)),
    "retention 3 x 20 x 12": ("parallel", _parallel(_window(1, 1, 8, 8, 4, 2, _rot(2)), _retention(3, 20, 12, [0.5, 1.0, 0.97], _rot(20)), 0.1, 2.0)),
    "retention 2 x 128 x 64": ("parallel", _parallel(_window(1, 1, 8, 8, 4, 2, _rot(2)), _retention(2, 128, 64, [0.99, 0.7], _rot(64)), 0.1, 2.0)),
    "mlstm 2 x 16 x 24": ("mlstm", _mlstm(2, 16, 24, 8.0)),
    "mlstm 3 x 20 x 12": ("mlstm", _mlstm(3, 20, 12, 15.0)),
    "mlstm 4 x 128 x 64": ("mlstm", _mlstm(4, 128, 64, 4.0)),
}


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", list(MIXERS))
def test_one_mixer_alone_in_every_cut(tmp_path, name, dtype):
    """A model of one layer without feed-forward: the mixer between an embedding and the head."""
    kind, mixer = MIXERS[name]
    cfg = _config(120, 96, [_layer(kind, mixer, None)])
    folder = write_folder(str(tmp_path / "one"), cfg, make_weights(cfg, len(name), mild=dtype == "bfloat16"))
    reqs = _requests(120, [70, 45, 137, 33, 1, 58, 2, 3], seed=5)
    _all_cuts(folder, dtype, reqs, plain_logits(folder, reqs), 16, 384, TOL[dtype], name)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_a_state_that_remembers_a_token_hundreds_of_positions_back(tmp_path, dtype):
    """Decays of 1 and near 1, forget gates that stay open: a token changed 400 positions back moves the last logits."""
    cfg = _config(90, 32, [_layer("parallel", _parallel(_window(2, 1, 8, 8, 12, 4, _rot(4)), _retention(2, 16, 16, [1.0, 0.998], _rot(4))), None),
                           _layer("mlstm", _mlstm(2, 16, 16, 15.0), None)])
    w = make_weights(cfg, 12, mild=dtype == "bfloat16")
    w["l1.mix.f.b"] = torch.tensor([9.0, 12.0], dtype=torch.bfloat16)
    folder = write_folder(str(tmp_path / "long"), cfg, w)
    wd = plain_kosusun.read_model(folder)[1]
    n = 430
    toks = random_prompt(90, n, 2)
    other = list(toks)
    other[30] = (toks[30] + 1) % 90
    want, moved = plain_kosusun.forward(cfg, wd, toks), plain_kosusun.forward(cfg, wd, other)
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
def test_all_cuts_match_plain(folders, mild_folders, name, dtype):
    folder = (mild_folders if dtype == "bfloat16" else folders)[name]
    reqs = _requests(SMALL[name][0]["vocab"], [70, 45, 197, 33, 1, 58, 2, 3], seed=5)
    _all_cuts(folder, dtype, reqs, plain_logits(folder, reqs), SMALL[name][1], 384, TOL[dtype], name)


def test_token_by_token_from_the_first(folders):
    for name in ("A", "B"):
        folder = folders[name]
        reqs = _requests(SMALL[name][0]["vocab"], [60], seed=21)
        want = plain_logits(folder, reqs)
        steps = trace_prefill_then_decode(reqs, tail=59)
        got = collect(steps, _replay(_runner(folder, "float32", 64, SMALL[name][1]), steps))
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


def test_bfloat16_through_the_plain_kernels_does_not_depend_on_the_cut(mild_folders):
    """Through the plain kernels a row's arithmetic is the same whatever stands beside it (no portion here is long
    enough for segments): bfloat16 logits are the same to the recurrences' last bits in every cut, which would show a
    stale slot or a page used again however small the difference."""
    from tiny_llm_infer_amd.engine.loading import load_model
    from tiny_llm_infer_amd.engine.runner import ModelRunner
    from tiny_llm_infer_amd.kernels.ops import HipOps
    folder = mild_folders["A"]
    reqs = _requests(160, [70, 45, 97, 33, 1, 58], seed=15)
    results = []
    for steps in (trace_whole(reqs), trace_portions(reqs, seed=3), trace_mixed(reqs, max_tokens=256, seed=9)):
        ops = HipOps("cuda:0")
        ops.use_plain_kernels()
        model, _ = load_model(folder, "bfloat16", "cuda:0", max_model_len=512, ops=ops)
        runner = ModelRunner(model, model.env, page_size=16, num_pages=16, max_requests=4, max_batch_tokens=512)
        results.append(collect(steps, _replay(runner, steps)))
    for rid in reqs:
        # (the mLSTM's running maximum is added up in another order for another cut: a bfloat16 may fall to its neighbour)
        for other in results[1:]:
            assert np.abs(results[0][rid] - other[rid]).max() <= 0.03 * np.abs(results[0][rid]).max(), rid


def test_long_decoding_through_recorded_launches(mild_folders):
    """150 tokens decoded one by one for three requests at once (bfloat16: the steps are replayed from recordings): the
    window passes over decoded tokens, blocks of them are pooled and come into sight."""
    folder = mild_folders["R"]
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


def test_recorded_steps_equal_eager_steps(mild_folders):
    """The same decode steps replayed from recordings and run eagerly, many rows (products of every size class), with the
    program's own work between the replays."""
    folder = mild_folders["R"]
    reqs = _requests(320, [20 + i % 7 for i in range(40)], seed=9)
    outs = []
    for graphs in (True, False):
        runner = _runner(folder, "bfloat16", 40 * 64, 32, max_requests=40)
        runner.use_graphs = runner.use_graphs and graphs
        steps = [{"step": 0, "entries": [{"id": r, "tokens": t[:10], "want": []} for r, t in reqs.items()], "end": []}]
        for j in range(10, 20):
            steps.append({"step": len(steps), "entries": [{"id": r, "tokens": [t[j]], "want": [0]} for r, t in reqs.items()], "end": []})
        got = []
        from tiny_llm_infer_amd.engine.replay import Replayer
        rp = Replayer(runner)
        for st in steps:
            got.append(rp.run_step(st))
            torch.cuda.synchronize()
            torch.randn(1000, device="cuda").sum()
        assert (runner.graph_replays > 0) == graphs
        outs.append(got[1:])
    for a, b in zip(*outs):
        assert np.abs(a - b).max() <= 2e-2 * np.abs(b).max()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_greedy_generation_through_the_engine(folders, mild_folders, dtype):
    from tiny_llm_infer_amd.engine.llm_engine import LLMEngine
    from tiny_llm_infer_amd.sampling.params import SamplingParams
    folder = (mild_folders if dtype == "bfloat16" else folders)["A"]
    prompts = [random_prompt(160, n, 90 + n) for n in (4, 19, 30, 41)]
    eng = LLMEngine.from_folder(folder, dtype=dtype, max_model_len=128, page_size=16, num_kv_blocks=32, max_num_seqs=3,
                                max_num_batched_tokens=32)
    got = eng.generate(prompts, SamplingParams(max_tokens=10, ignore_eos=True))
    if dtype == "float32":
        assert [r.token_ids for r in got] == [plain_greedy(folder, p, 10) for p in prompts]
    else:
        # rounding may turn a close call: every token must be the plain implementation's choice or within
        # the rounding error of it, given the tokens before
        cfg, w = plain_kosusun.read_model(folder)
        for p, r in zip(prompts, got):
            logits = plain_kosusun.forward(cfg, w, p + r.token_ids)[len(p) - 1:-1]
            for z, t in zip(logits, r.token_ids):
                assert float(z.max() - z[t]) <= 2 * TOL["bfloat16"] * float(z.abs().max())
    eng.runner.cache.check()
    assert eng.runner.cache.free_pages() == eng.runner.cache.pages_per_group()


# ------------------------------------------------------------------ the command line ---
def test_the_programs_take_a_kosusun_folder(folders, tmp_path):
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
