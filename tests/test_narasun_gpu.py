"""The Narasun design on the GPU: every mechanism's kernel alone against the plain implementation's function, then the model
through the engine's step function, its replay tool and its generation loop, under every way of cutting and batching, in
32-bit and in bfloat16."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

import narasun_models as nm
import plain_narasun as pn
import traces
from conftest import ROOT, rel_err

pytestmark = pytest.mark.gpu

if torch.cuda.is_available():
    from inferflux_amd import SamplingParams
    from inferflux_amd.engine.api import load_runner
    from inferflux_amd.engine.context import StepContext, StepEntry
    from inferflux_amd.engine.engine import Engine
    from inferflux_amd.kernels import ops

DT = {"float32": torch.float32, "bfloat16": torch.bfloat16}
# Largest difference of a logit from the plain model's, relative to the largest logit.  32-bit: rounding over a few hundred
# operations.  bfloat16: the worst seen over these tests and half as much again; a key, a state, a sink, a bonus or a pass's
# input that is wrong moves a row by 10-100 %.  The rows of a sequence's first positions get more in bfloat16: a recurrent
# head's output is normed, so while its state holds one or a few outer products the output's direction hangs on single
# q . k products, which rounding q and k moves by a large fraction where they happen to be small.
TOL = {"float32": 4e-5, "bfloat16": 5e-2}
TOL_FIRST = {"float32": 4e-5, "bfloat16": 1e-1}
FIRST = 16
GAIN = {"float32": 2.0, "bfloat16": 1.0}
# The weights' seeds: ones with which no row of the sequences below hangs on a recurrent head whose output is nearly zero (there
# the exact model itself moves by 10 % when its normed rows are changed by half a unit in the last place of a bfloat16).
SEEDS = {"A": 43, "B": 44, "C": 42, "D": 43, "E": 44}
DEV = "cuda"


def rnd(seed, *shape, scale=1.0):
    return torch.randn(*shape, generator=torch.Generator().manual_seed(seed), dtype=torch.float64) * scale


def ids_of(seed, n, vocab):
    return torch.randint(0, vocab, (n,), generator=torch.Generator().manual_seed(seed)).tolist()


def T64(a):
    return torch.from_numpy(np.asarray(a, dtype=np.float64))


def N64(t):
    return t.double().cpu().numpy()


@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    """(configuration, precision) -> model folder.  The 32-bit runs take routers with random weights; the bfloat16 runs take
    models in which no choice of experts is a close call (``write_model``)."""
    out = {}
    for n in nm.CONFIGS:
        for dtype in DT:
            out[n, dtype] = nm.write_model(str(tmp_path_factory.mktemp(f"narasun{n}{dtype}")), nm.config(n), SEEDS[n], gain=GAIN[dtype],
                                           decisive_router=dtype == "bfloat16")
    return out


_PLAIN = {}


def plain(folder, ids, layers=False):
    if folder not in _PLAIN:
        _PLAIN[folder] = nm.load_plain(folder)
    key = (folder, tuple(ids), layers)
    if key not in _PLAIN:
        out = pn.forward(*_PLAIN[folder], list(ids), return_layers=layers)
        _PLAIN[key] = (T64(out[0]), T64(out[1])) if layers else T64(out)
    return _PLAIN[key]


def off(got, want, dtype, positions=None):
    """The rows' largest differences from ``want`` (relative to its largest entry) over what their positions allow: below 1 is
    within tolerance.  ``positions``: each row's place in its sequence (by default row i is position i)."""
    want = want.double()
    err = (got.double() - want).abs().amax(dim=1) / want.abs().max()
    positions = torch.arange(len(err)) if positions is None else torch.as_tensor(list(positions))
    allowed = torch.where(positions < FIRST, TOL_FIRST[dtype], TOL[dtype])
    rel_err(got, want)
    return float((err / allowed).max())


def run_whole(runner, rid, ids, want=None):
    runner.add_request(rid)
    out = runner.step([StepEntry(rid, ids, list(range(len(ids))) if want is None else want)]).cpu()
    runner.free_request(rid)
    return out


def _step_arrays(lens):
    q_len = torch.tensor(lens, dtype=torch.int32)
    q_start = torch.cumsum(q_len, 0).to(torch.int32) - q_len
    return q_start, q_len


def _row_req(lens):
    return torch.repeat_interleave(torch.arange(len(lens), dtype=torch.int32), torch.tensor(lens))


def _paged(k, v, dt, P=16, seed=5):
    """k [n, G, kd], v [n, G, dv] of one sequence in pages that lie anywhere in a pool: (K, V, block table [1, pages])."""
    n, G, kd = k.shape
    dv = v.shape[2]
    pages = -(-n // P)
    pool = pages + 3
    where = torch.randperm(pool, generator=torch.Generator().manual_seed(seed))[:pages]
    K = torch.zeros(pool, G, P, kd, dtype=dt)
    V = torch.zeros(pool, G, dv, P, dtype=dt)
    for j in range(n):
        K[where[j // P], :, j % P] = k[j].to(dt)
        V[where[j // P], :, :, j % P] = v[j].to(dt)
    return K.to(DEV), V.to(DEV), where.to(torch.int32)[None].contiguous().to(DEV)


# ---- each mechanism's kernel alone ------------------------------------------------------------
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("n,nH,nKV,d,dv", [(90, 4, 2, 16, 24), (200, 3, 3, 12, 12), (150, 3, 1, 10, 14), (260, 8, 2, 128, 128)])
def test_a_sink_per_head_joins_the_denominator(dtype, n, nH, nKV, d, dv):
    """Grouped heads without positions, a score per head that takes part in the softmax's sum alone; queries aimed at the
    sequence's first key, at the last key of a page and at the first of the next."""
    dt = DT[dtype]
    scale = 1.0 / d ** 0.5
    q, k, v = rnd(1, n, nH, d).to(dt).double(), rnd(2, n, nKV, d).to(dt).double(), rnd(3, n, nKV, dv).to(dt).double()
    sinks = torch.tensor([2.5, -1.0, 0.0, 4.0, -6.0, 1.0, 3.0, -2.0][:nH], dtype=torch.float32)
    for i in range(n):
        for h in range(nH):
            aim = (0, i - i % 16 - 1, i - i % 16, i)[(i + h) % 4]
            if aim >= 0:
                q[i, h] = (5.0 * k[aim, h // (nH // nKV)]).to(dt).double()
    K, V, table = _paged(k, v, dt)
    rows = torch.arange(n, dtype=torch.int32, device=DEV)
    zero = torch.zeros(n, dtype=torch.int32, device=DEV)
    want = np.stack([pn.causal_softmax(N64(q[:, h]) @ N64(k[:, h // (nH // nKV)]).T * scale, float(sinks[h])) @ N64(v[:, h // (nH // nKV)])
                     for h in range(nH)], axis=1).reshape(n, nH * dv)
    got = ops.attention_plain(q.to(dt).to(DEV), K, V, zero, rows, table, None, scale, sinks=sinks.to(DEV)).cpu()
    assert rel_err(got, T64(want)) < (2e-5 if dtype == "float32" else 2e-2)
    without = ops.attention_plain(q.to(dt).to(DEV), K, V, zero, rows, table, None, scale).cpu()
    assert rel_err(without, T64(want)) > 0.05


@pytest.mark.parametrize("d,qt", [(128, 2), (128, 1), (64, 2), (32, 1)])
@pytest.mark.parametrize("past,splits", [(0, 1), (0, 3), (130, 1), (130, 4)])
def test_sinks_in_the_tile_kernels(d, qt, past, splits):
    """A prompt's portion behind ``past`` keys through the kernels for tiles of rows (at head size 128 the tall tiles are the
    kernel that loads straight into LDS), whole and with the keys cut into splits; sinks from far below every score to above
    it, and rows whose one large score is for a key in the first split."""
    n, nH, nKV, P = 300, 4, 2, 16
    total = past + n
    q, k, v = rnd(1, n, nH, d).bfloat16().double(), rnd(2, total, nKV, d).bfloat16().double(), rnd(3, total, nKV, d).bfloat16().double()
    scale, sinks = d ** -0.5, torch.tensor([3.0, -40.0, 0.0, 12.0])
    for i in range(0, n, 7):
        q[i] = (4.0 * k[i % 11].repeat_interleave(nH // nKV, 0)).bfloat16().double()
    K, V, table = _paged(k, v, torch.bfloat16)
    i32 = lambda x: torch.tensor(x, dtype=torch.int32, device=DEV)
    rows = ops.attention_tile_rows(d, qt)
    q0 = list(range(0, n, rows))
    chunk = -(-(-(-total // splits)) // 64) * 64 if splits > 1 else 0
    out = torch.zeros(n, nH * d, dtype=torch.bfloat16, device=DEV)
    ops.attention_tiles(q.bfloat16().to(DEV), K, V, out, i32([0] * len(q0)), i32(q0), i32([0]), i32([n]), i32([total]), table, None, scale, qt, chunk,
                        splits, torch.arange(n, dtype=torch.int32, device=DEV), i32([0] * n), torch.arange(past, total, dtype=torch.int32, device=DEV),
                        sinks=sinks.to(DEV))
    full = np.concatenate([np.zeros((past, nH, d)), N64(q)])
    want = np.stack([pn.causal_softmax(full[:, h] @ N64(k[:, h // 2]).T * scale, float(sinks[h])) @ N64(v[:, h // 2]) for h in range(nH)], axis=1)
    want = want[past:].reshape(n, nH * d)
    assert rel_err(out.cpu(), T64(want)) < 2e-2
    heads = (out.cpu().double() - T64(want)).reshape(n, nH, d).abs().amax(dim=(0, 2)) / T64(want).reshape(n, nH, d).abs().amax(dim=(0, 2))
    assert float(heads.max()) < 3e-2        # (a head whose sink takes nearly everything has small outputs of its own)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("T,nH,nKV,d,dv", [(5, 4, 2, 16, 24), (200, 4, 2, 64, 64), (150, 3, 1, 10, 14), (130, 2, 2, 32, 16)])
def test_query_temperature_multiplies_the_queries_alone(dtype, T, nH, nKV, d, dv):
    dt, P = DT[dtype], 16
    qkv = rnd(1, T, (nH + nKV) * d + nKV * dv).to(dt)
    positions = torch.arange(3, 3 + T, dtype=torch.int32)
    mult = ops.query_temperature(positions.to(DEV), 0.7, 13)
    want_mult = pn.query_temperature(T + 3, {"coef": 0.7, "every": 13})[3:]
    assert rel_err(mult.cpu(), T64(want_mult)) < 1e-6 and bool(np.all((want_mult == 1.0) == (np.arange(3, 3 + T) < 12)))      # position 12 is the first of the next step
    pages = -(-T // P) + 1
    K = torch.zeros(pages, nKV, P, d, dtype=dt, device=DEV)
    V = torch.zeros(pages, nKV, dv, P, dtype=dt, device=DEV)
    slots = torch.arange(7, 7 + T, dtype=torch.int32, device=DEV)
    q = ops.rope_append(qkv.to(DEV), None, slots, None, None, ops.ROPE_NONE, 0, nH, nKV, d, K, V, P, dv, q_mult=mult).cpu()
    want = N64(qkv)[:, :nH * d].reshape(T, nH, d) * want_mult[:, None, None]
    assert rel_err(q, T64(want)) < (1e-6 if dtype == "float32" else 5e-3)
    flat_k = K.permute(0, 2, 1, 3).reshape(-1, nKV * d)[7:7 + T].cpu()
    flat_v = V.permute(0, 3, 1, 2).reshape(-1, nKV * dv)[7:7 + T].cpu()
    assert torch.equal(flat_k, qkv[:, nH * d:(nH + nKV) * d]) and torch.equal(flat_v, qkv[:, (nH + nKV) * d:])


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("H", [64, 100, 1030])
def test_mixes_with_the_row_before_over_steps(dtype, H):
    """Three requests in unequal portions, down to single rows: the row before a portion's first is the last of the request's
    last portion, zeros at its start; the kept rows lie behind a stretch of the slot that belongs to somebody else."""
    dt = DT[dtype]
    lens, slot, offset = {"a": 45, "b": 9, "c": 23}, {"a": 4, "b": 0, "c": 2}, 8
    data = {r: rnd(20 + i, n, H).to(dt) for i, (r, n) in enumerate(lens.items())}
    mu = torch.rand(3, H, generator=torch.Generator().manual_seed(1))
    state = torch.zeros(6, offset + H, dtype=torch.float32, device=DEV)
    at, got = {r: 0 for r in lens}, {r: [] for r in lens}
    for step in [{"a": 20, "b": 1, "c": 2}, {"c": 16, "a": 1}, {"b": 8, "a": 9, "c": 1}, {"a": 15, "c": 4}]:
        h = torch.cat([data[r][at[r]:at[r] + m] for r, m in step.items()])
        q_start, q_len = _step_arrays(list(step.values()))
        slots = torch.tensor([slot[r] for r in step], dtype=torch.int32)
        out = ops.shifted_mixes(h.to(DEV), mu.to(DEV), state, offset, _row_req(list(step.values())).to(DEV), q_start.to(DEV), q_len.to(DEV),
                                slots.to(DEV)).cpu()
        o = 0
        for r, m in step.items():
            got[r].append(out[:, o:o + m]); o += m; at[r] += m
    assert float(state[:, :offset].abs().max()) == 0 and float(state[[1, 3, 5]].abs().max()) == 0
    for r in lens:
        want = np.stack([pn.shifted_mix(N64(data[r]), N64(mu[s])) for s in range(3)])
        assert rel_err(torch.cat(got[r], dim=1), T64(want)) < (1e-6 if dtype == "float32" else 5e-3), r
        assert torch.equal(state[slot[r], offset:].cpu(), data[r][-1].float())


@pytest.mark.parametrize("wdtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("T,rank,C", [(1, 12, 48), (37, 5, 300), (130, 64, 512), (9, 128, 1024), (20, 3, 77)])
def test_the_decays_inner_product(wdtype, T, rank, C):
    a = rnd(1, T, rank + 7, scale=2.0).float()
    w = rnd(2, rank, C).to(DT[wdtype])
    got = ops.lowrank_tanh(a.to(DEV)[:, 7:], w.to(DEV)).cpu()
    assert rel_err(got, T64(np.tanh(N64(a)[:, 7:]) @ N64(w))) < 2e-6


def _time_mix_inputs(seed, T, H, d, dt):
    return [rnd(seed + i, T, H * d).to(dt) for i in range(4)] + [rnd(seed + 4, T, H * d, scale=1.5).float()]


def _time_mix_plain(r, k, v, g, z, w0, u, norm_w, eps, H, d):
    T = r.shape[0]
    heads = lambda x: N64(x).reshape(T, H, d)
    w = np.exp(-np.exp(N64(z) + N64(w0))).reshape(T, H, d)
    out = np.stack([pn.time_mix_recurrence(heads(r)[:, h], heads(k)[:, h], heads(v)[:, h], w[:, h], N64(u)[h]) for h in range(H)], axis=1)
    return pn.unit_rms(out, eps).reshape(T, H * d) * N64(norm_w) * pn.silu(N64(g))


@pytest.mark.parametrize("dtype", ["float32", "bfloat16", "float32 to bfloat16"])
@pytest.mark.parametrize("H,d", [(3, 16), (1, 12), (2, 10), (4, 64), (2, 128), (5, 40)])
def test_time_mix_over_steps_with_state_in_slots(dtype, H, d):
    """Three requests whose rows come in steps of unequal portions, their states in slots that lie anywhere behind a stretch
    of the row that belongs to somebody else, against each request's recurrence in one piece; in bfloat16 the long portions
    in chunks as well."""
    dt, out_dt = DT[dtype.split()[0]], DT[dtype.split()[-1]]
    eps, lens = 1e-5, {"a": 145, "b": 9, "c": 123}
    w0 = (-5.0 + 5.0 * torch.rand(H * d, generator=torch.Generator().manual_seed(8))).float()
    u, norm_w = rnd(9, H, d).float(), (1.0 + 0.3 * rnd(10, H * d)).float()
    data = {r: _time_mix_inputs(20 + 10 * i, n, H, d, dt) for i, (r, n) in enumerate(lens.items())}
    want = {r: _time_mix_plain(*x, w0, u, norm_w, eps, H, d) for r, x in data.items()}
    offset = 40
    for chunked in ((False, True) if dtype == "bfloat16" else (False,)):
        state = torch.zeros(6, offset + ops.gla_state_floats(H, d, d), dtype=torch.float32, device=DEV)
        slot = {"a": 4, "b": 0, "c": 2}
        at, got = {r: 0 for r in lens}, {r: [] for r in lens}
        for step in [{"a": 70, "b": 1, "c": 2}, {"c": 116, "a": 1}, {"b": 8, "a": 59, "c": 1}, {"a": 15, "c": 4}]:
            parts = [torch.cat([data[r][i][at[r]:at[r] + m] for r, m in step.items()]).to(DEV) for i in range(5)]
            q_start, q_len = _step_arrays(list(step.values()))
            slots = torch.tensor([slot[r] for r in step], dtype=torch.int32)
            chunks = ops.scan_chunks(q_start, q_len, 32, DEV) if chunked else None
            out = ops.time_mix_scan(*parts, w0.to(DEV), u.to(DEV), norm_w.to(DEV), eps, H, d, state, offset, q_start.to(DEV), q_len.to(DEV),
                                    slots.to(DEV), out_dt, chunks).cpu()
            assert out.dtype == out_dt
            o = 0
            for r, m in step.items():
                got[r].append(out[o:o + m]); o += m; at[r] += m
        assert float(state[:, :offset].abs().max()) == 0 and float(state[[1, 3, 5]].abs().max()) == 0     # nobody else's floats were touched
        for r in lens:
            assert at[r] == lens[r]
            assert rel_err(torch.cat(got[r]), T64(want[r])) < (2e-5 if dtype == "float32" else 2e-2), (r, chunked)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_a_key_far_back_is_still_in_time_mixings_state(dtype):
    """A channel that hardly decays is written at token 0 alone and read 700 tokens later, decoded one by one at the end: the
    read-out points along the value written then.  The bonus is off, so the token's own write says nothing."""
    dt, H, d, T = DT[dtype], 2, 32, 720
    r, k, v, g, z = [x.double() for x in _time_mix_inputs(3, T, H, d, dt)]
    k[:, 0] = 0.0
    k[0, :d] = 0.0
    k[0, 0] = 3.0
    r[T - 5:, :d] = 0.0
    r[T - 5:, 0] = 2.0
    z[:, 0] = -14.0
    parts = [x.to(dt) for x in (r, k, v, g)] + [z.float()]
    w0, u, norm_w = torch.zeros(H * d), torch.zeros(H, d), torch.ones(H * d)
    want = _time_mix_plain(*parts, w0, u, norm_w, 1e-6, H, d)
    state = torch.zeros(2, ops.gla_state_floats(H, d, d), dtype=torch.float32, device=DEV)
    got, p = [], 0
    for m in [300, 415, 1, 1, 1, 1, 1]:
        q_start, q_len = _step_arrays([m])
        chunks = ops.scan_chunks(q_start, q_len, 32, DEV) if m > 32 and dtype == "bfloat16" else None
        got.append(ops.time_mix_scan(*[x[p:p + m].to(DEV) for x in parts], w0.to(DEV), u.to(DEV), norm_w.to(DEV), 1e-6, H, d, state, 0,
                                     q_start.to(DEV), q_len.to(DEV), torch.tensor([1], dtype=torch.int32, device=DEV), dt, chunks).cpu())
        p += m
    got = torch.cat(got)
    assert rel_err(got[T - 5:], T64(want[T - 5:])) < (2e-5 if dtype == "float32" else 2e-2)
    read = N64(got)[T - 1, :d] / pn.silu(N64(parts[3])[T - 1, :d])
    v0 = N64(parts[2])[0, :d]
    assert float(read @ v0 / np.linalg.norm(read) / np.linalg.norm(v0)) > 0.999


def _memory_inputs(seed, T, H, d, dv, dt, gate_scale=3.0):
    """(rows [T, 2 H d + 2 H dv + 8 of something else], their columns, gates float [T, 2 H + 3], their columns)"""
    rows = torch.cat([rnd(seed, T, 8), rnd(seed + 1, T, 2 * H * d), rnd(seed + 2, T, 2 * H * dv)], dim=1).to(dt)
    gates = torch.cat([rnd(seed + 3, T, 3), rnd(seed + 4, T, 2 * H, scale=gate_scale)], dim=1).float()
    return rows, (8, 8 + H * d, 8 + 2 * H * d, 8 + 2 * H * d + H * dv), gates, (3, 3 + H)


def _memory_plain(rows, cols, gates, gate_cols, ib, fb, cap, norm_w, eps, H, d, dv):
    R, G, T = N64(rows), N64(gates), rows.shape[0]
    q = R[:, cols[0]:cols[0] + H * d].reshape(T, H, d) * d ** -0.5
    k = R[:, cols[1]:cols[1] + H * d].reshape(T, H, d)
    v = R[:, cols[2]:cols[2] + H * dv].reshape(T, H, dv)
    li = pn.soft_cap(G[:, gate_cols[0]:gate_cols[0] + H] + N64(ib), cap)
    lf = pn.log_sigmoid(pn.soft_cap(G[:, gate_cols[1]:gate_cols[1] + H] + N64(fb), cap))
    out = np.stack([pn.matrix_memory_recurrence(q[:, h], k[:, h], v[:, h], li[:, h], lf[:, h]) for h in range(H)], axis=1)
    return pn.unit_rms(out, eps).reshape(T, H * dv) * N64(norm_w) * pn.sigmoid(R[:, cols[3]:cols[3] + H * dv])


def _memory_call(rows, cols, gates, gate_cols, ib, fb, cap, norm_w, eps, H, d, dv, state, lens, slots, out_dt, chunked, single=False):
    q_start, q_len = _step_arrays(lens)
    chunks = ops.scan_chunks(q_start, q_len, ops.MEMORY_CHUNK, DEV) if chunked else None
    return ops.matrix_memory(rows.to(DEV), cols, gates.to(DEV), gate_cols, ib.to(DEV), fb.to(DEV), cap, norm_w.to(DEV), eps, H, d, dv, state,
                             q_start.to(DEV), q_len.to(DEV), torch.tensor(slots, dtype=torch.int32, device=DEV), _row_req(lens).to(DEV), out_dt,
                             single, chunks).cpu()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16", "float32 to bfloat16"])
@pytest.mark.parametrize("H,d,dv", [(4, 16, 24), (2, 12, 12), (3, 10, 14), (4, 64, 64), (1, 128, 256), (2, 256, 64), (2, 40, 200), (8, 32, 96), (5, 8, 8),
                                    (1, 300, 16)])
def test_matrix_memory_over_steps_with_state_in_slots(dtype, H, d, dv):
    """Three requests whose rows come in steps of unequal portions down to single tokens, their states in slots, against each
    request's recurrence in one piece; in bfloat16 in chunks on the matrix cores as well (portions that end inside a chunk,
    on its edge and just behind it)."""
    dt, out_dt = DT[dtype.split()[0]], DT[dtype.split()[-1]]
    eps, cap, lens = 1e-5, 9.0, {"a": 245, "b": 9, "c": 133}
    ib, fb = rnd(8, H).float(), (rnd(9, H) * 2 + 2).float()
    norm_w = (1.0 + 0.3 * rnd(10, H * dv)).float()
    data = {r: _memory_inputs(20 + 10 * i, n, H, d, dv, dt) for i, (r, n) in enumerate(lens.items())}
    want = {r: _memory_plain(*x, ib, fb, cap, norm_w, eps, H, d, dv) for r, x in data.items()}
    n_state = ops.matrix_memory_state_floats(H, d, dv)
    takes = ops.matrix_memory_takes_chunks(dt, d, dv)
    for chunked in ((False, True) if takes else (False,)):
        state = torch.zeros(6, n_state, dtype=torch.float32, device=DEV)
        slot = {"a": 4, "b": 0, "c": 2}
        at, got = {r: 0 for r in lens}, {r: [] for r in lens}
        for step in [{"a": 128, "b": 1, "c": 2}, {"c": 65, "a": 1}, {"a": 1, "b": 1, "c": 1}, {"b": 7, "a": 100, "c": 1}, {"a": 15, "c": 64}]:
            rows = torch.cat([data[r][0][at[r]:at[r] + m] for r, m in step.items()])
            gates = torch.cat([data[r][2][at[r]:at[r] + m] for r, m in step.items()])
            ms = list(step.values())
            single = max(ms) == 1
            out = _memory_call(rows, data["a"][1], gates, data["a"][3], ib, fb, cap, norm_w, eps, H, d, dv, state, ms, [slot[r] for r in step],
                               out_dt, chunked and not single, single)
            assert out.dtype == out_dt
            o = 0
            for r, m in step.items():
                got[r].append(out[o:o + m]); o += m; at[r] += m
        assert float(state[[1, 3, 5]].abs().max()) == 0     # nobody else's floats were touched
        for r in lens:
            assert at[r] == lens[r]
            assert rel_err(torch.cat(got[r]), T64(want[r])) < (3e-5 if dtype == "float32" else 2e-2), (r, chunked)


@pytest.mark.parametrize("H,d,dv", [(4, 64, 128), (2, 24, 40), (1, 256, 320)])
def test_chunks_on_the_matrix_cores_round_nothing_of_the_recurrence(H, d, dv):
    """From the same bfloat16 rows, with a float output, the chunks give what the 32-bit walk gives: the state, the weights
    and the sums are not rounded to 16 bits on their way through the matrix cores.  The states they leave agree too."""
    dt, cap, lens = torch.bfloat16, 15.0, [150, 1, 64, 200]
    ib, fb, norm_w = rnd(8, H).float(), (rnd(9, H) * 2 + 3).float(), torch.ones(H * dv)
    rows, cols, gates, gate_cols = _memory_inputs(3, sum(lens), H, d, dv, dt, gate_scale=5.0)
    outs, states = [], []
    for chunked in (False, True):
        state = torch.zeros(5, ops.matrix_memory_state_floats(H, d, dv), dtype=torch.float32, device=DEV)
        src = rows if chunked else rows.float()
        for _ in range(2):           # the second time from the states the first has left
            out = _memory_call(src, cols, gates, gate_cols, ib, fb, cap, norm_w, 1e-6, H, d, dv, state, lens, [3, 0, 4, 1], torch.float32, chunked)
        outs.append(out)
        states.append(state.cpu())
    assert rel_err(outs[1], outs[0]) < 2e-4
    assert rel_err(states[1], states[0]) < 2e-5


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_a_key_far_back_is_still_in_the_memory(dtype):
    """A head that hardly forgets is written strongly at token 0 along a key no later token comes near, and asked for it 700
    tokens later, decoded one by one at the end: the read-out points along the value written then.  The other head forgets."""
    dt, H, d, dv, T, cap = DT[dtype], 2, 32, 16, 720, 15.0
    rows, cols, gates, gate_cols = _memory_inputs(3, T, H, d, dv, dt, gate_scale=0.2)
    rows, gates = rows.double(), gates.double()
    rows[:, cols[0]] = 0.0                              # channel 0 of head 0's q and k belongs to the far key alone
    rows[:, cols[1]] = 0.0
    rows[0, cols[1]:cols[1] + d] = 0.0
    rows[0, cols[1]] = 3.0
    rows[T - 5:, cols[0]:cols[0] + d] = 0.0
    rows[T - 5:, cols[0]] = 2.0
    gates[0, gate_cols[0]] = 6.0
    gates[:, gate_cols[1]] = 12.0
    gates[:, gate_cols[1] + 1] = -2.0
    rows, gates = rows.to(dt), gates.float()
    ib, fb, norm_w = torch.zeros(H), torch.zeros(H), torch.ones(H * dv)
    want = _memory_plain(rows, cols, gates, gate_cols, ib, fb, cap, norm_w, 1e-6, H, d, dv)
    state = torch.zeros(2, ops.matrix_memory_state_floats(H, d, dv), dtype=torch.float32, device=DEV)
    got, p = [], 0
    for m in [300, 415, 1, 1, 1, 1, 1]:
        got.append(_memory_call(rows[p:p + m], cols, gates[p:p + m], gate_cols, ib, fb, cap, norm_w, 1e-6, H, d, dv, state, [m], [1], dt,
                                m > 1 and dtype == "bfloat16", m == 1))
        p += m
    got = torch.cat(got)
    assert rel_err(got[T - 5:], T64(want[T - 5:])) < (3e-5 if dtype == "float32" else 2e-2)
    read = N64(got)[T - 1, :dv] / pn.sigmoid(N64(rows)[T - 1, cols[3]:cols[3] + dv])
    v0 = N64(rows)[0, cols[2]:cols[2] + dv]
    assert float(read @ v0 / np.linalg.norm(read) / np.linalg.norm(v0)) > 0.999


@pytest.mark.parametrize("chunked", [False, True])
def test_gates_at_both_ends_of_their_cap(chunked):
    """Input gates at the cap and far below, forget gates that keep everything and that forget at once, in turns that reach
    across chunks: the running maximum jumps up at once and comes down with the forgetting."""
    H, d, dv, T, cap = 2, 16, 24, 200, 15.0
    rows, cols, gates, gate_cols = _memory_inputs(5, T, H, d, dv, torch.bfloat16)
    gates[:, gate_cols[0]:] = 0.0
    for t in range(T):
        gates[t, gate_cols[0]:gate_cols[0] + H] = 200.0 if t % 67 == 5 else (-200.0 if t % 3 else -20.0)
        gates[t, gate_cols[1]:gate_cols[1] + H] = -100.0 if t % 41 == 7 else (-1.0 if t % 5 else 8.0)
    ib, fb, norm_w = torch.tensor([0.5, -0.5]), torch.tensor([1.0, -1.0]), torch.ones(H * dv)
    want = _memory_plain(rows, cols, gates, gate_cols, ib, fb, cap, norm_w, 1e-6, H, d, dv)
    state = torch.zeros(1, ops.matrix_memory_state_floats(H, d, dv), dtype=torch.float32, device=DEV)
    got = _memory_call(rows, cols, gates, gate_cols, ib, fb, cap, norm_w, 1e-6, H, d, dv, state, [T], [0], torch.bfloat16, chunked)
    assert bool(torch.isfinite(got).all()) and rel_err(got, T64(want)) < 2e-2


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("T,E,top,K,ff", [(5, 6, 2, 64, 24), (70, 12, 2, 192, 64), (33, 3, 3, 100, 22), (90, 8, 1, 128, 32), (200, 30, 6, 256, 128)])
def test_experts_weighed_at_their_inputs(dtype, T, E, top, K, ff):
    """The sigmoid's scores choose and weigh, and the weight is on the expert's input: by the row kernels and, in bfloat16, by
    the grouped products on the matrix cores as well.  The inputs are large, so that the activation is far from linear."""
    dt = DT[dtype]
    p = "m"
    W = {f"{p}.router": rnd(1, E, K, scale=1.0 / K ** 0.5).to(dt).double()}
    for e in range(E):
        W[f"{p}.e{e}.gate"], W[f"{p}.e{e}.up"] = rnd(10 + e, ff, K, scale=2.0 / K ** 0.5).to(dt).double(), rnd(50 + e, ff, K, scale=2.0 / K ** 0.5).to(dt).double()
        W[f"{p}.e{e}.down"] = rnd(90 + e, K, ff, scale=1.0 / ff ** 0.5).to(dt).double()
    h = rnd(3, T, K).to(dt)
    Wn = {k: N64(v) for k, v in W.items()}
    want_ids, want_w = pn.route(N64(h), Wn, p, {"top": top})
    ids, weights = ops.moe_route(h.to(DEV), W[f"{p}.router"].to(dt).to(DEV), top)
    if dtype == "float32":
        assert np.array_equal(ids.cpu().numpy(), want_ids) and rel_err(weights.cpu(), T64(want_w)) < 1e-5
    ids_t, w_t = torch.from_numpy(want_ids.astype(np.int32)).to(DEV), torch.from_numpy(want_w).float().to(DEV)
    want = pn.moe(N64(h), Wn, p, {"router": {"top": top}})
    stack = lambda k: torch.stack([W[f"{p}.e{e}.{k}"].to(dt) for e in range(E)]).contiguous().to(DEV)
    gate, up, down = stack("gate"), stack("up"), stack("down")
    tol = 2e-5 if dtype == "float32" else 2e-2
    got = ops.moe_experts(h.to(DEV), gate, up, down, ids_t, w_t, weigh_input=True).cpu()
    assert rel_err(got, T64(want)) < tol
    assert rel_err(ops.moe_experts(h.to(DEV), gate, up, down, ids_t, w_t).cpu(), T64(want)) > 5 * tol     # (on the outputs it is another function)
    if dtype == "bfloat16" and ops.grouped_takes(dt, K, ff):
        paired = ops.pair_gate_up(gate, up)
        assert rel_err(ops.moe_experts_grouped(h.to(DEV), paired, down, ids_t, w_t, weigh_input=True).sum(torch.float32).cpu(), T64(want)) < tol
        assert rel_err(ops.moe_experts(h.to(DEV), paired, None, down, ids_t, w_t, weigh_input=True).cpu(), T64(want)) < tol


@pytest.mark.parametrize("H", [64, 100, 1030, 2048, 5120, 9000])
@pytest.mark.parametrize("out", ["float32", "bfloat16"])
def test_several_additions_in_the_norms_kernel(H, out):
    """Tensors of both types with factors, a product's partial sums and one vector for all rows, added in one kernel with the
    norm; picked rows leave the stream alone."""
    T, eps = 9, 1e-5
    x, w = rnd(1, T, H).float(), rnd(2, H).float()
    a, b, parts, vec = rnd(3, T, H).bfloat16(), rnd(4, T, H).float(), rnd(5, 3, T, H).float(), rnd(6, H).bfloat16()
    total = x.double() + 0.5 * a.double() - 2.0 * b.double() + parts.double().sum(0) + vec.double()
    want = pn.unit_rms(N64(total), eps) * N64(w)
    delta = ops.DeltaSum([(a.to(DEV), 0.5), (ops.ScaledDelta(b.to(DEV), 2.0), -1.0), (ops.SliceSums(parts.to(DEV), torch.bfloat16), 1.0), (vec.to(DEV), 1.0)])
    s = x.to(DEV)
    rows = torch.tensor([7, 0, 3], dtype=torch.int32, device=DEV)
    tol = 1e-5 if out == "float32" else 1e-2
    assert rel_err(ops.add_rmsnorm(s, delta, w.to(DEV), eps, DT[out], rows).cpu(), T64(want)[[7, 0, 3]]) < tol
    assert torch.equal(s.cpu(), x)
    assert rel_err(ops.add_rmsnorm(s, delta, w.to(DEV), eps, DT[out]).cpu(), T64(want)) < tol
    assert rel_err(s.cpu(), total) < 1e-6
    other = rnd(7, T, H).float()
    joined = ops.join_stream(x.to(DEV), delta, other.to(DEV), DT[out]).cpu()
    assert rel_err(joined[:, :H], total) < tol and rel_err(joined[:, H:], other) < tol
    assert torch.equal(ops.join_stream(x.to(DEV), None, other.to(DEV), torch.float32).cpu(), torch.cat([x, other], 1))


@pytest.mark.parametrize("M", [1, 7, 16, 17, 40, 64])
@pytest.mark.parametrize("block,tail,K", [(128, 16, 256), (256, 64, 520), (1024, 100, 1024), (48, 5, 64)])
def test_products_of_several_inputs_in_one_launch(M, block, tail, K):
    n = 4
    x = rnd(1, n + 1, M, K).bfloat16()
    w = rnd(2, n * block + tail, K, scale=K ** -0.5).bfloat16()
    lw = ops.prepare_linear(w.to(DEV), tile_rows=16)
    want = torch.cat([x[i].double() @ w[i * block:(i + 1) * block if i < n else None].double().t() for i in range(n + 1)], dim=1)
    if not ops.takes_blocks(M, lw, block):
        assert M > 16 and block % 128
        with pytest.raises(ops.KernelError):
            ops.linear_blocks(x.to(DEV), lw, block)
        return
    assert rel_err(ops.linear_blocks(x.to(DEV), lw, block, torch.float32).cpu(), want) < 1e-5
    assert rel_err(ops.linear_blocks(x.to(DEV), lw, block).cpu(), want) < 1e-2
    for i in range(n + 1):                  # a part of a weight is a weight of its own
        part = lw.part(i * block, (i + 1) * block if i < n else n * block + tail)
        assert rel_err(ops.linear(x[i].to(DEV), part, torch.float32).cpu(), want[:, i * block:(i + 1) * block if i < n else None]) < 1e-5


# ---- the model through the engine -----------------------------------------------------------------
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", list(nm.CONFIGS))
def test_whole_prompts(name, dtype, folders):
    folder, vocab = folders[name, dtype], nm.CONFIGS[name]["vocab"]
    runner = load_runner(folder, DT[dtype], num_pages=32, max_requests=2)
    for seed, n in ((1, 1), (2, 2), (3, 37), (4, 200)):
        ids = ids_of(seed, n, vocab)
        assert off(run_whole(runner, "w", ids), plain(folder, ids), dtype) < 1, (name, n)
    runner.manager.check()


@pytest.mark.parametrize("name", ["A", "B", "C", "D"])
def test_stream_after_every_layer(name, folders):
    folder = folders[name, "float32"]
    runner = load_runner(folder, torch.float32, num_pages=8)
    ids = ids_of(3, 50, nm.CONFIGS[name]["vocab"])
    _, streams = plain(folder, ids, layers=True)
    runner.add_request("p")
    runner.manager.reserve("p", len(ids))
    ctx = StepContext([StepEntry("p", ids, [0])], runner.manager, torch.float32, runner.device)
    model = runner.model
    assert len(model.plan.schedule) == streams.shape[0]
    x, pending = model.embedding.forward(ctx), None
    embedded = x.clone()
    for i, e in enumerate(model.plan.schedule):
        if e.before is not None:
            x, pending = model.injections[e.before].apply(x, pending, ctx, embedded)
        x, pending = model.blocks[e.layer].forward(x, pending, ctx, runner.storage.binding(i))
        after = x + ops.DeltaSum.of(pending).tensor(x)
        assert rel_err(after.cpu(), streams[i]) < 1e-5, i


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("kind", ["recurrent_only", "parallel_only", "ranks_from_the_tensors"])
def test_models_without_pages_and_with_open_sizes(kind, dtype, tmp_path):
    """A model of matrix memories alone keeps no pages at all; one of paired mixers alone; a config that leaves the decays'
    ranks to the tensors' shapes."""
    layers = {
        "recurrent_only": [nm.layer(nm.memory(2, 16, 16, 5.0), nm.moe(4, 2, 24)), nm.layer(nm.memory(1, 24, 40, 9.0, "mlstm_2"), None)],
        "parallel_only": [nm.layer(nm.parallel(nm.attention(4, 4, 16, 16, 0.3, 0.3, 9), nm.time_mix(2, 16, 8), 0.5, 0.5), nm.moe(4, 1, 24)),
                          nm.layer(nm.parallel(nm.attention(2, 1, 16, 8, 0.3), nm.time_mix(3, 8, 1), 1.0, 2.0), None)],
        "ranks_from_the_tensors": [nm.layer(nm.parallel(nm.attention(2, 2, 32, 32, 0.2, 0.2, 64), nm.time_mix(2, 32, 11), 0.9, 1.1), nm.moe(8, 8, 16)),
                                   nm.layer(nm.memory(2, 32, 32, 7.0), nm.dense(48))],
    }[kind]
    cfg = nm.model(150, 64, 1e-5, layers, loop=(0, 2, 2) if kind == "recurrent_only" else None)
    folder = nm.write_model(str(tmp_path / "m"), cfg, 9, gain=GAIN[dtype], decisive_router=dtype == "bfloat16",
                            keep_rank=kind != "ranks_from_the_tensors")
    runner = load_runner(folder, DT[dtype], num_pages=20, max_requests=3)
    assert len(runner.manager.groups) == {"recurrent_only": 0, "parallel_only": 1, "ranks_from_the_tensors": 1}[kind]
    ids = ids_of(8, 230, 150)
    want = plain(folder, ids)
    assert off(run_whole(runner, "w", ids), want, dtype) < 1
    runner.add_request("c")
    runner.add_request("o")
    rows, p = [], 0
    for m in [2, 100, 1, 1, 64, 3, 1, 58]:
        rows.append(runner.step([StepEntry("o", ids_of(p, 2, 150), []), StepEntry("c", ids[p:p + m], list(range(m)))]).cpu())
        p += m
    assert p == len(ids) and off(torch.cat(rows), want, dtype) < 1
    runner.manager.check()


def test_first_tokens(folders):
    """Position 0 sees itself and its sink, a zero state, zeros before it and a maximum of 0: its logits are a function of the
    token."""
    folder = folders["D", "float32"]
    runner = load_runner(folder, torch.float32, num_pages=8)
    for tok in (0, 77, 98):
        a, b = run_whole(runner, "x", [tok]), run_whole(runner, "y", [tok, 5, 9, 2])
        assert rel_err(a, plain(folder, [tok])) < TOL["float32"] and rel_err(a[0], b[0]) < 2e-6
        assert rel_err(b, plain(folder, [tok, 5, 9, 2])) < TOL["float32"]


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", list(nm.CONFIGS))
def test_prefill_against_decoding_and_portions(name, dtype, folders):
    folder, vocab = folders[name, dtype], nm.CONFIGS[name]["vocab"]
    runner = load_runner(folder, DT[dtype], num_pages=24, max_requests=4)
    ids = ids_of(31, 170, vocab)
    want = plain(folder, ids)
    whole = run_whole(runner, "w", ids)
    runner.add_request("d")                                      # token by token from the first
    single = torch.cat([runner.step([StepEntry("d", [t], [0])]).cpu() for t in ids])
    runner.free_request("d")
    runner.add_request("c")                                      # portions of changing size, down to two tokens and one
    rows, p = [], 0
    for m in [2, 3, 16, 2, 1, 31, 2, 64, 17, 2, 30]:
        rows.append(runner.step([StepEntry("c", ids[p:p + m], list(range(m)))]).cpu())
        p += m
    runner.free_request("c")
    assert p == len(ids)
    for got in (whole, single, torch.cat(rows)):
        assert off(got, want, dtype) < 1
    if dtype == "float32":      # in 32-bit a row's arithmetic does not depend on the cutting, beyond rounding
        assert rel_err(single, whole) < 1e-5 and rel_err(torch.cat(rows), whole) < 1e-5
    runner.manager.check()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["A", "C", "D"])
def test_unequal_requests_in_one_batch_against_each_alone(name, dtype, folders):
    folder, vocab = folders[name, dtype], nm.CONFIGS[name]["vocab"]
    runner = load_runner(folder, DT[dtype], num_pages=40, max_requests=4)
    seqs = {"a": ids_of(41, 90, vocab), "b": ids_of(42, 23, vocab), "c": ids_of(43, 140, vocab), "d": ids_of(44, 2, vocab)}
    for r in seqs:
        runner.add_request(r)
    at = {r: 0 for r in seqs}
    got = {r: [] for r in seqs}
    plan = [{"a": 30, "b": 2, "c": 64, "d": 1}, {"a": 1, "c": 40, "d": 1}, {"a": 17, "b": 20, "c": 1}, {"a": 1, "b": 1, "c": 1},
            {"a": 41, "c": 34}]
    for step in plan:
        entries = [StepEntry(r, seqs[r][at[r]:at[r] + m], list(range(m))) for r, m in step.items()]
        out = runner.step(entries).cpu()
        o = 0
        for r, m in step.items():
            got[r].append(out[o:o + m]); o += m; at[r] += m
    for r, ids in seqs.items():
        assert at[r] == len(ids)
        assert off(torch.cat(got[r]), plain(folder, ids), dtype) < 1, r
        if dtype == "float32":      # in 32-bit a row's arithmetic depends neither on the cutting nor on its neighbours, beyond rounding
            runner.free_request(r)
            assert rel_err(torch.cat(got[r]), run_whole(runner, r + "'", ids)) < 1e-5, r


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_long_decoding_keeps_its_pages_and_its_state(dtype, folders):
    folder = folders["A", dtype]
    runner = load_runner(folder, DT[dtype], num_pages=30, max_requests=2)
    ids = ids_of(51, 420, 300)
    want = plain(folder, ids)
    runner.add_request("d")
    got = [runner.step([StepEntry("d", ids[:9], [8])]).cpu()[0]]
    for p in range(9, len(ids)):
        got.append(runner.step([StepEntry("d", [ids[p]], [0])]).cpu()[0])
    assert off(torch.stack(got), want[8:], dtype, range(8, len(ids))) < 1
    runner.manager.check()
    assert runner.graph_replays > 0          # decode steps of a model with state of its own are replayed graphs too


def test_a_freed_slot_starts_from_zero_state(folders):
    """The same prompt gives the same logits in a slot and pages that another request has just used."""
    folder = folders["B", "float32"]
    runner = load_runner(folder, torch.float32, num_pages=6, max_requests=1)
    a, b = ids_of(52, 80, 131), ids_of(53, 61, 131)
    first = run_whole(runner, "a", a)
    run_whole(runner, "b", b)
    assert torch.equal(run_whole(runner, "a2", a), first)
    folder = folders["A", "float32"]
    runner = load_runner(folder, torch.float32, num_pages=12, max_requests=2)
    a, b = ids_of(54, 80, 300), ids_of(55, 61, 300)
    first = run_whole(runner, "a", a)
    runner.add_request("b")
    runner.step([StepEntry("b", b, [])])
    runner.add_request("a2")
    out = runner.step([StepEntry("a2", a, list(range(len(a))))]).cpu()
    runner.free_request("b")
    assert rel_err(out, first) < 1e-5 and rel_err(run_whole(runner, "a3", a), first) < 1e-5


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", list(nm.CONFIGS))
def test_replay_of_traces_with_pages_and_slots_used_again(name, dtype, folders, tmp_path):
    """Through bin/trace_run as a user would: whole, prefill then decode, portions, and mixed steps of up to four live
    requests, one process, a pool so small that pages and slots are used again."""
    folder, vocab = folders[name, dtype], nm.CONFIGS[name]["vocab"]
    seqs = {f"r{i}": ids_of(60 + i, n, vocab) for i, n in enumerate([45, 150, 1, 96, 33, 260, 64])}
    all_steps, expected, offset = [], {}, 0
    for build in (traces.whole, traces.prefill_then_decode, traces.portions, lambda s: traces.mixed(s, seed=7)):
        steps, exp = build(seqs)
        for s in steps:
            s["step"] += offset
        expected.update({k + offset: v for k, v in exp.items()})
        all_steps += steps
        offset += len(steps)
    out = str(tmp_path / "out")
    proc = subprocess.Popen([sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model", folder, "--dtype", dtype, "--out", out,
                             "--max-tokens", str(traces.peak_tokens(all_steps))], stdin=subprocess.PIPE, stdout=subprocess.PIPE, text=True)
    try:
        for s in all_steps:
            proc.stdin.write(json.dumps(s) + "\n")
            proc.stdin.flush()
            assert proc.stdout.readline().strip() == f"done {s['step']}"
        proc.stdin.close()
        assert proc.wait(timeout=120) == 0
    finally:
        if proc.poll() is None:
            proc.kill()
    assert sorted(int(f[:-4]) for f in os.listdir(out)) == sorted(expected)
    for step, rows in expected.items():
        got = torch.from_numpy(np.fromfile(os.path.join(out, f"{step}.f32"), dtype="<f4").reshape(len(rows), vocab))
        want = torch.stack([plain(folder, seqs[rid])[p] for rid, p in rows])
        assert off(got, want, dtype, [p for _, p in rows]) < 1, (step, rows[:3])


def _drawn_config(seed):
    """A configuration drawn from sizes of every kind: heads of many and few channels, grouped and ungrouped, values wider and
    narrower than keys, temperatures that step at every token, around a page's size or not at all, ranks and factors, one
    expert and all of them, layers in any order with and without feed-forward, loops anywhere."""
    import random
    rng = random.Random(seed)
    width = rng.choice([48, 72, 96, 160])
    layers = []
    for _ in range(rng.choice([1, 2, 3, 4])):
        if rng.random() < 0.5:
            mixer = nm.memory(rng.choice([1, 2, 3, 5]), rng.choice([6, 8, 16, 20, 32, 64, 128]), rng.choice([8, 10, 16, 32, 64, 136]),
                              rng.choice([2.0, 6.0, 15.0]), rng.choice(["mlstm", "mlstm_2"]))
        else:
            kv = rng.choice([1, 2, 3])
            dim = rng.choice([8, 12, 16, 32, 48, 64, 96])
            left = nm.attention(kv * rng.choice([1, 2, 4]), kv, dim, rng.choice([dim, 8, 10, 16, 32, 64]), rng.choice([1.0, 2.0]) / dim ** 0.5,
                                *rng.choice([(None, None), (0.3, 1), (0.5, 16), (0.2, 17), (1.0, 64), (-0.2, 5)]))
            right = nm.time_mix(rng.choice([1, 2, 3]), rng.choice([8, 10, 16, 32, 64]), rng.choice([1, 4, 9, 32]))
            mixer = nm.parallel(left, right, rng.choice([1.0, 0.5, 1.5]), rng.choice([1.0, 0.3, 2.0]))
        mlp = rng.choice([None, nm.dense(64), nm.dense(50), nm.moe(4, 2, 24), nm.moe(8, 1, 16), nm.moe(3, 3, 40), nm.moe(6, 4, 32)])
        layers.append(nm.layer(mixer, mlp))
    n = len(layers)
    loop = None
    if rng.random() < 0.6:
        start = rng.randrange(n)
        loop = (start, rng.randrange(start + 1, n + 1), rng.choice([1, 2, 3]))
    return nm.model(rng.choice([61, 128, 500]), width, rng.choice([1e-5, 1e-6, 1e-3]), layers, loop=loop)


@pytest.mark.parametrize("seed", range(14))
def test_drawn_configurations(seed, tmp_path):
    """Whole prompts, portions and decoding of drawn configurations against the plain implementation, both precisions."""
    cfg = _drawn_config(seed)
    for dtype in ("float32", "bfloat16"):
        folder = nm.write_model(str(tmp_path / dtype), cfg, 80 + seed, gain=GAIN[dtype], decisive_router=dtype == "bfloat16")
        runner = load_runner(folder, DT[dtype], num_pages=24, max_requests=3)
        ids = ids_of(seed, 150, cfg["vocab"])
        want = plain(folder, ids)
        assert off(run_whole(runner, "w", ids), want, dtype) < 1, (seed, dtype, cfg)
        runner.add_request("c")
        runner.add_request("other")
        rows, p = [], 0
        for m in [33, 2, 64, 1, 1, 17, 1, 1, 1, 29]:
            out = runner.step([StepEntry("other", ids_of(p, 3, cfg["vocab"]), []), StepEntry("c", ids[p:p + m], list(range(m)))]).cpu()
            rows.append(out)
            p += m
        assert p == len(ids) and off(torch.cat(rows), want, dtype) < 1, (seed, dtype, cfg)
        runner.manager.check()


# ---- generation through the engine's own entry point and scheduler ------------------------------
@pytest.mark.parametrize("name", ["A", "C"])
def test_greedy_generation_through_the_engine(name, folders):
    folder, vocab = folders[name, "float32"], nm.CONFIGS[name]["vocab"]
    cfg, W = nm.load_plain(folder)
    prompts = [ids_of(70 + i, n, vocab) for i, n in enumerate([5, 40, 1, 77, 19, 130])]
    want = [pn.greedy_generate(cfg, W, p, 10) for p in prompts]
    engine = Engine.load(folder, dtype="float32", kv_pages=64, max_batch_size=4, chunked_prefill_tokens=32, prefill_tokens_alone=48)
    outs = engine.generate(prompts, SamplingParams(temperature=0.0, max_tokens=10, ignore_eos=True))
    assert [o.token_ids for o in outs] == want
    assert engine.runner.graph_replays > 0                       # decode steps ran as replayed graphs
    folder = folders[name, "bfloat16"]
    cfg, W = nm.load_plain(folder)
    engine = Engine.load(folder, dtype="bfloat16", kv_pages=64, max_batch_size=4, chunked_prefill_tokens=32)
    outs = engine.generate(prompts, SamplingParams(temperature=0.0, max_tokens=10, ignore_eos=True))
    for p, o in zip(prompts, outs):        # bfloat16 may pick another token where two logits nearly tie
        full = pn.forward(cfg, W, p + o.token_ids)
        for i, tok in enumerate(o.token_ids):
            row = full[len(p) - 1 + i]
            assert row[tok] >= row.max() - 0.08 * np.abs(row).max(), (name, i)


def test_completion_from_the_command_line(folders, capsys):
    from inferflux_amd import cli
    folder = folders["B", "float32"]
    cfg, W = nm.load_plain(folder)
    prompt = ids_of(90, 21, 131)
    assert cli.main(["completion", "--model", folder, "--prompt-ids", ",".join(map(str, prompt)), "--max-tokens", "7", "--temperature", "0",
                     "--ignore-eos", "--dtype", "float32", "--kv-pages", "32", "--max-parallel-sequences", "2"]) == 0
    said = capsys.readouterr().out
    want = pn.greedy_generate(cfg, W, prompt, 7)
    assert str(want)[1:-1].replace(" ", "") in said.replace(" ", ""), (want, said)
