"""The Vugotar decoder in the engine against the plain implementation (tests/plain_vugotar.py): every mechanism alone
through its kernels, then whole models of small odd sizes through the step function, the cache manager, the replayer's
schedules and the engine's own entry point."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

import plain_vugotar as plain
import vugotar_cases as cases
from helpers import replay, schedule_mixed, schedule_portions, schedule_tail_singly, schedule_whole, tokens_needed

pytestmark = pytest.mark.gpu
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
DEV = "cuda:0"


def dev(a, dtype=torch.float32):
    return torch.as_tensor(np.asarray(a), dtype=dtype).to(DEV).contiguous()


def bf16_grid(a):
    return torch.from_numpy(np.asarray(a, dtype=np.float64)).to(torch.bfloat16).double().numpy()


def i32(a):
    return torch.tensor(list(a), dtype=torch.int32, device=DEV)


class Runs:
    """The arrays a kernel reads of a step: one run (first position, rows, state slot) per sequence, packed one after another."""

    def __init__(self, runs):
        counts = [n for _, n, _ in runs]
        pos = [p for first, n, _ in runs for p in range(first, first + n)]
        self.rows, self.seqs, self.max_run, self.limits = sum(counts), len(runs), max(counts), None
        self.row_seq, self.positions = i32([s for s, n in enumerate(counts) for _ in range(n)]), i32(pos)
        self.ctx_lens = i32([p + 1 for p in pos])
        self.run_start = i32(np.concatenate([[0], np.cumsum(counts)]))
        self.seq_start, self.seq_end = i32([f for f, _, _ in runs]), i32([f + n for f, n, _ in runs])
        self.state_slots = i32([s for _, _, s in runs])


# ------------------------------------------------------------------------------ mechanisms alone
def test_the_stream_with_its_terms_and_norm():
    """x += sum of factor * term + a constant row, + the embedding again; the norm whose weight is stored around zero; rows
    gathered for the head; terms as tensors and as the slices of a split product."""
    from kvcm_amd import ops
    rng = np.random.default_rng(0)
    for T, H in ((5, 48), (3, 321), (2, 4100), (2, 9004)):      # the last two: rows kept in registers, and rows too long for that
        x, again, bias, w = rng.normal(size=(T, H)) * 2, rng.normal(size=(T, H)), rng.normal(size=H), 0.3 * rng.normal(size=H)
        ys = rng.normal(size=(3, T, H))
        for n, factors, use_bias, use_again, splits in ((0, (), False, False, 1), (1, (1.0,), True, False, 3), (2, (0.7, -1.5), False, True, 1),
                                                        (3, (1.0, 2.0, 0.25), True, True, 5), (0, (), False, True, 1)):
            want = x + sum((f * y for f, y in zip(factors, ys)), np.zeros((T, H)))
            want = want + (bias if use_bias else 0.0) + (again if use_again else 0.0)
            normed = plain.offset_norm(want, w, 1e-5)
            terms = []
            for i, f in enumerate(factors):
                if i % 2 == 0 and splits > 1:
                    parts = rng.normal(size=(splits, T, H))
                    parts[0] = ys[i] - parts[1:].sum(0)
                    terms.append((ops.PartialSums(dev(parts), splits, T, H, torch.empty(T, H, device=DEV)), f))
                else:
                    terms.append((dev(ys[i]), f))
            add = ops.StreamTerms(terms, dev(bias) if use_bias else None)
            for dt, tol in ((torch.float32, 1e-5), (torch.bfloat16, 2.0 ** -7)):
                xs, out = dev(x), torch.empty(T, H, dtype=dt, device=DEV)
                ops.stream_terms(xs, 1e-5, add=add, again=dev(again) if use_again else None, weight=dev(1.0 + w), out=out)
                np.testing.assert_allclose(xs.cpu().numpy(), want, atol=3e-6 * np.abs(want).max() * splits ** 0.5, err_msg=f"{T}x{H} n={n}")
                np.testing.assert_allclose(out.float().cpu().numpy(), normed, atol=tol * np.abs(normed).max(), err_msg=f"{T}x{H} n={n} {dt}")
                rows = [T - 1, 0, T - 1]
                xs, out = dev(x), torch.empty(3, H, dtype=dt, device=DEV)
                ops.stream_terms(xs, 1e-5, add=add, again=dev(again) if use_again else None, weight=dev(1.0 + w), out=out, rows=i32(rows))
                np.testing.assert_allclose(out.float().cpu().numpy(), normed[rows], atol=tol * np.abs(normed).max())
                assert torch.equal(xs, dev(x))
    with pytest.raises(ValueError, match="4 terms"):
        ops.stream_terms(dev(x), 1e-5, add=ops.StreamTerms([(dev(x), 1.0)] * 4), weight=dev(w), out=torch.empty(T, H, device=DEV))


@pytest.mark.parametrize("shape", [dict(nh=4, nkv=2, d=16, dv=12, rot=8), dict(nh=3, nkv=1, d=10, dv=10, rot=10), dict(nh=2, nkv=2, d=128, dv=64, rot=64),
                                   dict(nh=1, nkv=1, d=70, dv=6, rot=0)])
@pytest.mark.parametrize("halves", [False, True])
def test_rotation_then_a_norm_per_head_without_a_weight(shape, halves):
    from kvcm_amd import ops
    nh, nkv, d, dv, rot = (shape[k] for k in ("nh", "nkv", "d", "dv", "rot"))
    rng = np.random.default_rng(d + nh)
    B, eps, base = 8, 1e-5, 700.0
    pos = [0, 1, 7, 8, 100, 1000, 5000, 3]
    T = len(pos)
    proj = rng.normal(size=(T, (nh + nkv) * d + nkv * dv + 5))
    q, k = proj[:, :nh * d].reshape(T, nh, d), proj[:, nh * d:(nh + nkv) * d].reshape(T, nkv, d)
    v = proj[:, (nh + nkv) * d:(nh + nkv) * d + nkv * dv].reshape(T, nkv, dv)

    def turned(x):
        if not rot:
            return x
        if not halves:
            return plain.rotate_pairs(x, pos, rot, base)
        order = np.arange(rot).reshape(2, -1).T.reshape(-1)      # pairs (i, i + rot/2) laid out as neighbours, and back
        y = x.copy()
        y[..., order] = plain.rotate_pairs(x[..., order], pos, rot, base)
        return y

    want_q, want_k = plain.rms(turned(q), eps), plain.rms(turned(k), eps)
    table = torch.empty(T, max(rot, 2), device=DEV)
    if rot:
        ops.rotary_pairs_table(i32(pos), table, rot, base)
    slots = i32([17, 3, 9, 0, 31, 8, 1, -1])
    for dt, tol in ((torch.float32, 2e-5), (torch.bfloat16, 2.0 ** -7)):
        q_out = torch.empty(T, nh * d, dtype=dt, device=DEV)
        kc, vc = torch.zeros(4, nkv, B, d, dtype=dt, device=DEV), torch.zeros(4, nkv, dv, B, dtype=dt, device=DEV)
        ops.head_norm_store(dev(proj), q_out, nh, nkv, d, dv, eps, plain_norm=True, cos_sin=table if rot else None, rot=rot, halves=halves,
                            slots=slots, kcache=kc, vcache=vc)
        np.testing.assert_allclose(q_out.float().cpu().numpy(), want_q.reshape(T, -1), atol=tol * np.abs(want_q).max())
        for t, s in enumerate(slots.tolist()):
            if s >= 0:
                np.testing.assert_allclose(kc[s // B, :, s % B].float().cpu().numpy(), want_k[t], atol=tol * np.abs(want_k).max())
                np.testing.assert_allclose(vc[s // B, :, :, s % B].float().cpu().numpy(), v[t], atol=tol * np.abs(v).max())
        assert int(kc.float().abs().sum((1, 3)).gt(0).sum()) == T - 1      # the row without a slot stored nothing


def _paged(rng, k, v, B, dtype, passed):
    """Keys [n, G, d] and values [n, G, dv] of one sequence on shuffled pages, rubbish (NaN) everywhere else; the sequence's
    first ``passed`` pages are given back (table entry -1)."""
    n, G, d = k.shape
    dv = v.shape[2]
    pages = -(-n // B)
    ids = rng.permutation(pages + 5)[:pages]
    kh = np.full((pages + 5, G, B, d), np.nan)
    vh = np.full((pages + 5, G, dv, B), np.nan)
    for t in range(passed * B, n):
        kh[ids[t // B], :, t % B] = k[t]
        vh[ids[t // B], :, :, t % B] = v[t]
    return dev(kh, dtype), dev(vh, dtype), [-1 if i < passed else int(p) for i, p in enumerate(ids)]


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("shape", [dict(nh=4, nkv=2, d=16, dv=16, B=16, C=20), dict(nh=3, nkv=1, d=32, dv=24, B=8, C=33), dict(nh=2, nkv=2, d=10, dv=14, B=8, C=0),
                                   dict(nh=2, nkv=1, d=64, dv=64, B=16, C=1), dict(nh=6, nkv=2, d=128, dv=128, B=32, C=70), dict(nh=4, nkv=1, d=24, dv=16, B=16, C=64),
                                   dict(nh=2, nkv=2, d=64, dv=40, B=16, C=150), dict(nh=1, nkv=1, d=64, dv=130, B=16, C=48)])
def test_chunked_attention_with_a_sink_and_keys_that_stand_out_at_every_edge(shape, dtype):
    """One key is made to dominate the scores of the last row; it is put far away, at page borders, at the first position, just
    inside and just outside the last row's chunk; decoded rows and runs of rows, through shuffled pages with rubbish in the
    others and with the pages of passed chunks given back."""
    from kvcm_amd import ops
    s = shape
    nh, nkv, d, dv, B, C = (s[k] for k in ("nh", "nkv", "d", "dv", "B", "C"))
    rng = np.random.default_rng(nh * 100 + d + C)
    n, scale, factor = 230, 0.1, 0.8
    last = n - 1
    spots = {0, B - 1, 2 * B, last - 1, last, 64, 63, 128}
    if C:
        edge = last // C * C
        spots |= {edge, edge - 1, edge + 1, edge - C, edge - C - 1}
    pos = np.arange(n)
    for spot in sorted(p for p in spots if 0 <= p <= last):
        k, v, q = rng.normal(size=(n, nkv, d)), rng.normal(size=(n, nkv, dv)), rng.normal(size=(n, nh, d))
        k[spot] *= 4.0
        q[last] = np.repeat(k[spot], nh // nkv, axis=0) * 1.5
        if dtype == torch.bfloat16:
            k, v, q = bf16_grid(k), bf16_grid(v), bf16_grid(q)
        want = plain.chunk_attention(q, k, v, scale, pos, pos, C) * factor
        tol = 3e-5 if dtype == torch.float32 else 3e-2
        for first in (last, last - 9, 100, 0):
            passed = first // C * C // B if C else 0      # pages wholly before the chunk of the run's first row
            kc, vc, table = _paged(rng, k, v, B, dtype, passed)
            st = Runs([(first, n - first, 0)])
            tables = i32(table)
            out = torch.full((n - first, nh * dv + 6), 7.0, dtype=dtype, device=DEV)      # a view into wider rows, as a joined layer hands it over
            qd = dev(q[first:].reshape(n - first, -1), dtype)
            rule = dict(chunk=C, sink=True, out_scale=factor)
            ops.attention_window_pool(qd, out[:, 3:3 + nh * dv], kc, vc, None, None, tables, len(table), st.row_seq, st.ctx_lens, nh, nkv, d, dv, scale,
                                      0, 0, **rule)
            np.testing.assert_allclose(out[:, 3:3 + nh * dv].float().cpu().numpy(), want[first:].reshape(n - first, -1), atol=tol, err_msg=f"key {spot} rows from {first}")
            assert float((out[:, :3].float() - 7.0).abs().max()) == 0.0 and float((out[:, 3 + nh * dv:].float() - 7.0).abs().max()) == 0.0
            if ops.attention_window_pool_tiles_supported(d, dv, dtype, B):
                out2 = torch.empty(n - first, nh * dv + 6, dtype=dtype, device=DEV)
                ops.attention_window_pool_tiles(qd, out2[:, 3:3 + nh * dv], kc, vc, None, None, tables, len(table), st.run_start, st.seq_start, 1, n - first,
                                                nh, nkv, d, dv, scale, 0, 0, **rule)
                np.testing.assert_allclose(out2[:, 3:3 + nh * dv].float().cpu().numpy(), want[first:].reshape(n - first, -1), atol=tol,
                                           err_msg=f"tiles: key {spot} rows from {first}")


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_the_sink_takes_most_of_the_weight_where_scores_are_low(dtype):
    """Scores far below zero: an ordinary softmax still adds up to one, here nearly all goes to the sink; and scores far above,
    where it must not overflow."""
    from kvcm_amd import ops
    rng = np.random.default_rng(1)
    n, d, dv, B, C = 90, 32, 32, 16, 40
    v = rng.normal(size=(n, 1, dv)) + 2.0
    for level in (-6.0, 0.0, 90.0):
        k = np.zeros((n, 1, d))
        k[:, 0, 0] = 1.0
        q = np.zeros((n, 1, d))
        q[:, 0, 0] = level
        vv = bf16_grid(v)
        want = plain.chunk_attention(q, k, vv, 1.0, np.arange(n), np.arange(n), C)
        kc, vc, table = _paged(rng, k, vv, B, dtype, 0)
        st = Runs([(0, n, 0)])
        tol = 2e-5 if dtype == torch.float32 else 2e-2
        out = torch.empty(n, dv, dtype=dtype, device=DEV)
        ops.attention_window_pool(dev(q[:, 0], dtype), out, kc, vc, None, None, i32(table), len(table), st.row_seq, st.ctx_lens, 1, 1, d, dv, 1.0, 0, 0,
                                  chunk=C, sink=True)
        np.testing.assert_allclose(out.float().cpu().numpy(), want[:, 0], atol=tol)
        if dtype == torch.bfloat16:
            ops.attention_window_pool_tiles(dev(q[:, 0], dtype), out, kc, vc, None, None, i32(table), len(table), st.run_start, st.seq_start, 1, n, 1, 1, d, dv,
                                            1.0, 0, 0, chunk=C, sink=True)
            np.testing.assert_allclose(out.float().cpu().numpy(), want[:, 0], atol=tol)
        if level < 0:
            assert np.abs(want).max() < 0.4      # where an ordinary softmax would give about 2


def _state_inputs(rng, T, heads, groups, dk, dv):
    q, k, v = rng.normal(size=(T, groups, dk)), rng.normal(size=(T, groups, dk)), rng.normal(size=(T, heads, dv))
    a, b = rng.normal(size=(T, heads)), 2 * rng.normal(size=(T, heads))
    return q, k, v, a, b, 0.5 * rng.normal(size=heads) - 1.0, 0.7 * rng.normal(size=heads) - 2.0, rng.normal(size=heads)


def _state_want(delta, q, k, v, a, b, dt_bias, a_log, skip):
    dt = plain.softplus(a + dt_bias)
    if not delta:
        return plain.state_space(v, k, q, dt, a_log, skip)
    return plain.gated_delta(plain.unit(q) * q.shape[2] ** -0.5, plain.unit(k), v, np.exp(-np.exp(a_log) * dt), plain.logistic(b))


@pytest.mark.parametrize("delta", [True, False])
@pytest.mark.parametrize("shape", [(4, 2, 12, 20), (3, 1, 32, 8), (2, 2, 64, 40), (1, 1, 5, 3), (4, 4, 96, 17), (2, 1, 130, 33), (1, 1, 256, 16)])
def test_states_with_one_decay_per_head_over_runs_cut_at_random(shape, delta):
    """Two sequences of unequal length, their runs interleaved in steps and cut at random, slots that held rubbish; once every step
    walked row by row, once in pieces of 8 rows."""
    from kvcm_amd import ops
    heads, groups, dk, dv = shape
    rng = np.random.default_rng(sum(shape))
    lens = (75, 50)
    data = [_state_inputs(rng, n, heads, groups, dk, dv) for n in lens]
    for d in data[1:]:
        d[5][:], d[6][:], d[7][:] = data[0][5], data[0][6], data[0][7]      # the model's constants are the same for both
    want = [_state_want(delta, *d) for d in data]
    top = max(np.abs(w).max() for w in want)
    for piece in (None, 8):
        state = torch.full((4, heads, dk, dv), 3.0e4, device=DEV)
        done, got = [0, 0], [np.zeros((n, heads * dv)) for n in lens]
        while any(d < n for d, n in zip(done, lens)):
            runs, take = [], []
            for s in rng.permutation(2):
                n = min(int(rng.choice([1, 1, 2, 9, 30])), lens[s] - done[s])
                if n:
                    runs.append((done[s], n, (3, 1)[s]))
                    take.append((s, done[s], n))
                    done[s] += n
            st = Runs(runs)
            pack = lambda i: dev(np.concatenate([data[s][i][p:p + n].reshape(n, -1) for s, p, n in take]))
            o = torch.empty(st.rows, heads * dv, device=DEV)
            carry = None
            if piece:
                carry = torch.full((ops.gated_state_carry_floats(st.rows, st.seqs, heads, dk, dv, delta, piece),), float("nan"), device=DEV)
            extra = dict(b=pack(4)) if delta else dict(d_skip=dev(data[0][7]))
            ops.gated_state(pack(0), pack(1), pack(2), pack(3), dev(data[0][5]), dev(data[0][6]), o, state, st, heads, groups, dk, dv, carry=carry,
                            piece=piece, **extra)
            r = 0
            for s, p, n in take:
                got[s][p:p + n] = o[r:r + n].cpu().numpy()
                r += n
        for s in range(2):
            np.testing.assert_allclose(got[s], want[s].reshape(lens[s], -1), atol=1e-5 * top * (1 if delta else 3), err_msg=f"sequence {s} pieces of {piece}")


@pytest.mark.parametrize("delta", [True, False])
def test_a_token_written_hundreds_of_rows_ago_comes_back_through_every_piece(delta):
    """The state as a lookup: one key, orthogonal to all others, is written at row 3 and asked for at the last of 700 rows, across
    pieces of the kernels' own size, from a slot and from nothing."""
    from kvcm_amd import ops
    rng = np.random.default_rng(2)
    T, heads, dk, dv = 700, 2, 32, 24
    q, k, v, a, b, dt_bias, a_log, skip = _state_inputs(rng, T, heads, 1, dk, dv)
    k[:, :, 0] = 0.0
    k[3], q[-1] = 0.0, 0.0
    k[3, 0, 0] = q[-1, 0, 0] = 1.0
    a_log[:] = -9.0      # hardly any decay
    skip[:] = 0.0
    b[3] = 9.0
    want = _state_want(delta, q, k, v, a, b, dt_bias, a_log, skip)
    assert all(np.abs(want[-1, h]).max() > 0.1 and np.corrcoef(want[-1, h], v[3, h])[0, 1] > 0.95 for h in range(heads))
    top = np.abs(want).max()
    for cut in (0, 2, 150):
        state = torch.full((2, heads, dk, dv), float("nan"), device=DEV)
        rows = []
        for lo, hi in ((0, cut), (cut, T)):
            if lo == hi:
                continue
            st = Runs([(lo, hi - lo, 1)])
            o = torch.empty(hi - lo, heads * dv, device=DEV)
            carry = torch.full((ops.gated_state_carry_floats(hi - lo, 1, heads, dk, dv, delta),), float("nan"), device=DEV)
            part = lambda x: dev(x[lo:hi].reshape(hi - lo, -1))
            extra = dict(b=part(b)) if delta else dict(d_skip=dev(skip))
            ops.gated_state(part(q), part(k), part(v), part(a), dev(dt_bias), dev(a_log), o, state, st, heads, 1, dk, dv, carry=carry, **extra)
            rows.append(o.cpu().numpy())
        np.testing.assert_allclose(np.concatenate(rows), want.reshape(T, -1), atol=2e-5 * top, err_msg=f"cut at {cut}")
        assert not torch.isnan(state[1]).any() and torch.isnan(state[0]).all()


def test_gates_norms_and_routing_alone():
    """The gate before a norm over groups, a silu gate after a norm per head, biases and a row gate at the gated activation, a
    factor on the routing weights."""
    from kvcm_amd import ops
    rng = np.random.default_rng(6)
    for T, groups, size in ((5, 3, 16), (2, 1, 50), (3, 2, 700), (2, 2, 5000)):
        y, z, w = rng.normal(size=(T, groups * size)), rng.normal(size=(T, groups * size + 4)) * 2, 1 + 0.2 * rng.normal(size=groups * size)
        want = plain.rms((y * plain.silu(z[:, :groups * size])).reshape(T, groups, size), 1e-5).reshape(T, -1) * w
        for dt, tol in ((torch.float32, 1e-5), (torch.bfloat16, 2.0 ** -7)):
            out = torch.zeros(T, groups * size + 3, dtype=dt, device=DEV)
            ops.group_norm_gate(dev(y), dev(z), dev(w), out[:, 1:1 + groups * size], groups, size, 1e-5)
            np.testing.assert_allclose(out[:, 1:1 + groups * size].float().cpu().numpy(), want, atol=tol * np.abs(want).max())
            assert not out[:, 0].any() and not out[:, 1 + groups * size:].any()
    T, heads, d, I = 7, 3, 20, 37
    o, g, w = rng.normal(size=(T, heads * d)), rng.normal(size=(T, heads * d)) * 2, 1 + 0.2 * rng.normal(size=d)
    for act, fn in (("silu", plain.silu), ("sigmoid", plain.logistic)):
        out = torch.empty(T, heads * d, device=DEV)
        ops.head_norm_gate(dev(o), dev(g), dev(np.tile(w, heads)), out, heads, d, 1e-5, activation=act)
        np.testing.assert_allclose(out.cpu().numpy(), (plain.rms(o.reshape(T, heads, d), 1e-5) * w).reshape(T, -1) * fn(g), atol=2e-5)
    gu, bias, rg = rng.normal(size=(T, 2 * I + 3)), rng.normal(size=2 * I), rng.normal(size=(T, 4)) * 3
    for use_bias in (False, True):
        for use_gate in (False, True):
            z = gu[:, :2 * I] + (bias if use_bias else 0.0)
            want = plain.silu(z[:, :I]) * z[:, I:] * (plain.logistic(rg[:, 2:3]) if use_gate else 1.0)
            for dt, tol in ((torch.float32, 1e-6), (torch.bfloat16, 2.0 ** -7)):
                out = torch.empty(T, I + 5, dtype=dt, device=DEV)
                ops.gated_act(dev(gu), out[:, 2:2 + I], "silu", bias=dev(bias) if use_bias else None, row_gate=dev(rg)[:, 2:] if use_gate else None)
                np.testing.assert_allclose(out[:, 2:2 + I].float().cpu().numpy(), want, atol=tol * 10)
    for E, top, factor in ((8, 4, 2.5), (5, 1, 0.3), (1, 1, 1.0), (70, 6, 1.7)):
        z = rng.normal(size=(9, E)) * 2
        want_c, want_w = plain.choose_experts(z, top, factor)
        chosen, weight = torch.empty(9, top, dtype=torch.int32, device=DEV), torch.empty(9, top, device=DEV)
        ops.moe_route(dev(z), E, top, chosen, weight, over_chosen=True, factor=factor)
        assert chosen.cpu().numpy().tolist() == want_c.tolist()
        np.testing.assert_allclose(weight.cpu().numpy(), want_w, atol=3e-6 * factor)


class Alone(Runs):
    """A step as a part on its own sees it."""

    def __init__(self, runs, ops, dtype):
        super().__init__(runs)
        self.ops, self.dtype, self.buffers, self.shared, self.tune_products = ops, dtype, {}, {}, None

    def ws(self, name, shape, dtype=None):
        dtype = dtype or self.dtype
        fill = float("nan") if dtype.is_floating_point else -1
        return self.buffers.setdefault((name, shape[1], dtype), torch.full(shape, fill, dtype=dtype, device=DEV))

    def flat(self, name, numel, dtype=torch.float32):
        return self.buffers.setdefault((name, numel), torch.empty(numel, dtype=dtype, device=DEV))

    def scratch(self, name, rows, n, k):
        return None


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_sublayers_run_on_their_own_and_joined(dtype):
    """The parts beside their joined form: a feed-forward with biases, experts with a gated shared one, and the state mixers run by
    themselves give what the plain functions give, and so does the joined layer of them."""
    from kvcm_amd import ops
    from kvcm_amd.parts.base import BuildContext, PartSpec
    from kvcm_amd.parts.joined_parts import JoinedSublayers
    from kvcm_amd.registry import FEED_FORWARDS, MIXERS
    rng = np.random.default_rng(9)
    H, T, eps = 40, 21, 1e-5
    h = bf16_grid(rng.normal(size=(T, H)))
    specs = {
        "delta": ("mixer", PartSpec("gated_delta", {"heads": 4, "kv_heads": 2, "dim": 12, "vdim": 10, "conv": 3, "eps": eps}, "d.")),
        "space": ("mixer", PartSpec("state_space_duality", {"heads": 3, "vdim": 8, "state": 14, "groups": 1, "norm_groups": 2, "conv": 2, "eps": eps}, "s.")),
        "dense": ("ffn", PartSpec("gated_mlp", {"intermediate_size": 24, "bias": True}, "f.")),
        "experts": ("ffn", PartSpec("routed_experts", {"experts": 5, "top": 2, "ff": 12, "routing": "softmax_chosen", "route_factor": 1.8, "activation": "silu_gated",
                                                       "shared": PartSpec("gated_mlp", {"intermediate_size": 20}, "e.shared."), "shared_gate": "shared.sg"}, "e."))}
    context = lambda: BuildContext(dtype, torch.device(DEV), H, 16, ops)
    tensors, every = {}, {}

    def bind(part):
        for p in [part] + [s for s in part.sub_parts()]:
            for sub in list(p.sub_parts()) if p is not part else []:
                bind(sub)
            bound = {}
            for ps in p.param_specs():
                for name, shape in ps.sources:
                    if name not in tensors:
                        a = rng.normal(size=shape) * (shape[-1] ** -0.5 if len(shape) == 2 else 0.3) + (1.0 if ps.role == "vector" else 0.0)
                        tensors[name] = bf16_grid(a)
                stored = torch.float32 if ps.role in ("vector", "bias") else dtype
                bound[ps.name] = torch.cat([dev(tensors[n], stored) for n, _ in ps.sources], 0)
            p.bind(bound)
        return part

    def states(part):
        for name, need in part.cache_needs().items():
            class Slots:
                def __init__(self, need):
                    self.t = torch.full((2,) + need.shape, float("nan"), device=DEV)

                def slots(self, index):
                    return self.t
            part.attach_named_cache(name, Slots(need), 0)

    def total(value):
        terms = ops.StreamTerms.of(value)
        x = torch.zeros(T, H, device=DEV)
        ops.stream_terms(x, eps, add=terms)
        return x.cpu().numpy()

    m = {n: s.params for n, (_, s) in specs.items()}
    for name, (registry, spec) in specs.items():
        part = bind((MIXERS if registry == "mixer" else FEED_FORWARDS).get(spec.kind)(spec.params, spec.prefix, context()))
        states(part)
        every[name] = total(part.forward(Alone([(0, T, 1)], ops, dtype), dev(h, dtype)))
    t = tensors
    want = {"delta": plain.delta_mixer(h, t, "d.", m["delta"], eps), "space": plain.mamba2_mixer(h, t, "s.", m["space"], eps), "dense": plain.dense_ff(h, t, "f."),
            "experts": plain.mixture(h, t, "e.", {"router": {"top": 2, "scale": 1.8}, "shared": {"ff": 20}})}
    tol = 2e-5 if dtype == torch.float32 else 4e-2
    for name in specs:
        np.testing.assert_allclose(every[name], want[name], atol=tol * max(1.0, np.abs(want[name]).max()), err_msg=name)
    for members, factors in ((("delta", "space", "experts"), (0.6, -1.4, 1.0)), (("space", "delta", "dense"), (1.0, 2.0, 1.0))):
        listed = tuple((n, specs[n][0], PartSpec(specs[n][1].kind, {**m[n], **({"out_factor": f} if specs[n][0] == "mixer" else {})}, specs[n][1].prefix))
                       for n, f in zip(members, factors))
        part = bind(JoinedSublayers({"members": listed}, "l.", context()))
        for member in part.members:
            states(member)
        got = total(part.forward(Alone([(0, T, 1)], ops, dtype), dev(h, dtype)))
        joined = sum(f * want[n] for n, f in zip(members, factors))
        np.testing.assert_allclose(got, joined, atol=tol * max(1.0, np.abs(joined).max()), err_msg=str(members))


# ------------------------------------------------------------------------------ whole models
LENGTHS = (150, 41, 7, 1, 90, 23)


@pytest.fixture(scope="module")
def models():
    made = {}

    def get(name, dtype):
        if (name, dtype) not in made:
            from kvcm_amd.engine.replay import TraceReplayer
            raw = cases.CONFIGS[name]
            cfg, tensors = cases.tensors_for(raw, seed=len(name) + sum(map(ord, name)))
            reqs = cases.requests_for(raw, LENGTHS, seed=3)
            t = cases.as_numpy(tensors)
            ref = {rid: plain.forward(raw, t, toks) for rid, toks in reqs.items()}
            rp = TraceReplayer(None, dtype, max_tokens=tokens_needed(reqs, 3), block_size=cases.BLOCK_SIZE[name], max_live=3,
                               architecture="Vugotar", model_config=cfg, tensors=tensors)
            made[(name, dtype)] = (rp, reqs, ref, raw, t)
        return made[(name, dtype)]
    return get


def errors(got, ref):
    """Per position: the root mean square over the vocabulary of the difference (means taken off) over the logits' own spread."""
    spread = np.sqrt(np.mean([np.var(r, axis=1).mean() for r in ref.values()]))
    out = {}
    for rid in ref:
        d = got[rid].astype(np.float64) - ref[rid]
        e = np.sqrt(np.var(d, axis=1)) / spread
        assert not np.isnan(e).any(), f"{rid}: positions without logits"
        out[rid] = e
    return out


# float32 is the sharp test: every position within 1e-4 of the logits' spread and 5e-6 on average.  In bfloat16 the inputs of
# every product and the pages are rounded to 8 bits: the mean error is held and at most one position in fifty lies beyond a fifth.
def within(got, ref, dtype, what=""):
    e = errors(got, ref)
    every = np.concatenate(list(e.values()))
    if dtype == "float32":
        rid = max(e, key=lambda r: e[r].max())
        assert every.max() <= 1e-4, f"{what}: request {rid} position {int(e[rid].argmax())} is off by {every.max():.3g} of the logits' spread"
        assert every.mean() <= 5e-6, f"{what}: the mean error is {every.mean():.3g} of the logits' spread"
    else:
        assert every.mean() <= 0.03, f"{what}: the mean error is {every.mean():.3g} of the logits' spread"
        assert (every > 0.2).mean() <= 0.02, f"{what}: {(every > 0.2).sum()} of {every.size} positions are off by more than a fifth"


CASES = [(n, d) for n in cases.CONFIGS for d in ("float32", "bfloat16")]


def check(models, case, make_steps):
    rp, reqs, ref, _, _ = models(*case)
    got = replay(rp, make_steps(reqs), reqs)
    within(got, ref, case[1], str(case))
    assert all(rp.core.blocks_in_use(g) == 0 for g in range(rp.core.num_groups))
    return got


@pytest.mark.parametrize("name", list(cases.CONFIGS))
def test_layer_by_layer_against_the_plain_stream(models, name):
    """The residual stream after every layer of a whole prompt in 32-bit."""
    rp, reqs, _, raw, t = models(name, "float32")
    toks = reqs["r1"]
    trace = []
    plain.forward(raw, t, toks, trace)
    model = rp.runner.model
    seen = []
    for block in model.blocks:
        original = block.forward

        def wrapped(step, x, pending, original=original):
            out = original(step, x, pending)      # what the layer adds is still pending: added to a copy here
            ops, stream = model.ctx.ops, x.clone()
            ops.stream_terms(stream, 1e-5, add=out)
            seen.append(stream[:len(toks)].cpu().numpy())
            return out
        block.forward = wrapped
    try:
        rp.step({"step": 0, "entries": [{"id": "a", "tokens": toks, "want": [0]}], "end": ["a"]})
    finally:
        for block in model.blocks:
            del block.forward
    assert len(seen) == len(trace) == len(model.blocks)
    for i, (g, w) in enumerate(zip(seen, trace)):
        np.testing.assert_allclose(g, w, atol=2e-5 * max(1.0, np.abs(w).max()), err_msg=f"after layer {i}")


@pytest.mark.parametrize("case", CASES)
def test_whole_prompts(models, case):
    check(models, case, schedule_whole)


@pytest.mark.parametrize("case", CASES)
def test_prompt_then_token_by_token(models, case):
    check(models, case, lambda reqs: schedule_tail_singly(reqs, tail=80))


@pytest.mark.parametrize("case", CASES)
def test_portions_down_to_two_tokens(models, case):
    check(models, case, schedule_portions)
    check(models, case, lambda reqs: schedule_portions(reqs, sizes=(2, 2, 3, 1, 2, 40, 2)))


@pytest.mark.parametrize("case", CASES)
@pytest.mark.parametrize("seed", [0, 1])
def test_unequal_requests_in_one_batch_on_reused_pages(models, case, seed):
    check(models, case, lambda reqs: schedule_mixed(reqs, seed=seed, max_live=3))


@pytest.mark.parametrize("name", list(cases.CONFIGS))
def test_32bit_logits_do_not_depend_on_cut_batch_or_pages(models, name):
    rp, reqs, _, _, _ = models(name, "float32")
    whole = replay(rp, schedule_whole(reqs), reqs)
    for steps in (schedule_tail_singly(reqs, tail=80), schedule_portions(reqs), schedule_mixed(reqs, seed=2, max_live=3)):
        other = replay(rp, steps, reqs)
        for rid in reqs:
            np.testing.assert_allclose(other[rid], whole[rid], atol=2e-5, rtol=0)


@pytest.mark.parametrize("case", [("P", "float32"), ("Q", "bfloat16"), ("R", "bfloat16"), ("S", "float32")])
def test_steps_replayed_from_recorded_launch_lists(models, case):
    """Every part says it is capturable: a step's shape is recorded once as a list of launches and replayed with only the
    step's metadata changed; padding rows and padding sequences must leave the pages alone."""
    from kvcm_amd.engine.replay import TraceReplayer
    _, reqs, ref, raw, _ = models(*case)
    cfg, tensors = cases.tensors_for(raw, seed=len(case[0]) + sum(map(ord, case[0])))
    rp = TraceReplayer(None, case[1], max_tokens=tokens_needed(reqs, 3), block_size=cases.BLOCK_SIZE[case[0]], max_live=3,
                       architecture="Vugotar", model_config=cfg, tensors=tensors, use_programs=True)
    assert rp.programs is not None
    for steps in (schedule_mixed(reqs, seed=5, max_live=3), schedule_tail_singly(reqs, tail=20)):
        within(replay(rp, steps, reqs), ref, case[1], str(case))
    assert rp.steps_replayed > 50


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["P", "Q", "R", "S"])
def test_long_decoding_far_beyond_every_chunk(name, dtype):
    """300 tokens one by one: every chunk ends and begins among decoded tokens, states carry on; pages of passed chunks are
    given back, an attention without chunks keeps everything."""
    from kvcm_amd.engine.replay import TraceReplayer
    raw = cases.CONFIGS[name] if dtype == "float32" else cases.with_every_expert_chosen(cases.CONFIGS[name])
    cfg, tensors = cases.tensors_for(raw, seed=1 + ord(name))
    n = 300
    toks = cases.requests_for(raw, (n,), seed=11)["r0"]
    ref = {"r0": plain.forward(raw, cases.as_numpy(tensors), toks)}
    steps = [{"step": 0, "entries": [{"id": "r0", "tokens": toks[:4], "want": [0, 1, 2, 3]}], "end": []}]
    steps += [{"step": i, "entries": [{"id": "r0", "tokens": [toks[i]], "want": [0]}], "end": []} for i in range(4, n)]
    rp = TraceReplayer(None, dtype, max_tokens=320, block_size=cases.BLOCK_SIZE[name], max_live=2, architecture="Vugotar",
                       model_config=cfg, tensors=tensors)
    within(replay(rp, steps, {"r0": toks}), ref, dtype, name)
    B = cases.BLOCK_SIZE[name]
    tables = rp.tables()["r0"]
    for g, spec in enumerate(rp.core.groups):
        if spec.kind == "state":
            continue
        first_needed = n // spec.chunk * spec.chunk // B if spec.chunk else 0
        assert [p >= 0 for p in tables[g]] == [i >= first_needed for i in range(len(tables[g]))], (g, spec)
    rp.step({"step": n, "entries": [], "end": ["r0"]})


def test_a_short_request_on_a_long_request_s_pages_and_slot(models):
    rp, _, _, raw, t = models("P", "float32")
    long_, short = cases.requests_for(raw, (150, 5), seed=21).values()
    rp.step({"step": 0, "entries": [{"id": "a", "tokens": long_, "want": []}], "end": ["a"]})
    got = rp.step({"step": 1, "entries": [{"id": "b", "tokens": short, "want": list(range(5))}], "end": ["b"]})
    ref = plain.forward(raw, t, short)
    np.testing.assert_allclose(got, ref, atol=3e-5 * np.abs(ref).max())


def test_the_first_tokens_of_a_sequence(models):
    """Positions 0, 1, 2 alone and one by one: chunks, rotations, convolutions and states at their start."""
    for name in cases.CONFIGS:
        rp, _, _, raw, t = models(name, "float32")
        toks = cases.requests_for(raw, (3,), seed=31)["r0"]
        ref = plain.forward(raw, t, toks)
        rows = [rp.step({"step": i, "entries": [{"id": "f", "tokens": [toks[i]], "want": [0]}], "end": ["f"] if i == 2 else []})[0] for i in range(3)]
        np.testing.assert_allclose(np.stack(rows), ref, atol=3e-5 * np.abs(ref).max(), err_msg=name)


def test_a_prompt_long_enough_to_be_walked_in_pieces():
    """Runs of 512 rows and more take the recurrences' piece-by-piece walk: a prompt in one step, and cut so that one portion takes
    the pieces and the others do not."""
    from kvcm_amd.engine.replay import TraceReplayer
    raw = cases.CONFIGS["U"]
    cfg, tensors = cases.tensors_for(raw, seed=14)
    n = 620
    toks = cases.requests_for(raw, (n,), seed=12)["r0"]
    ref = plain.forward(raw, cases.as_numpy(tensors), toks)
    for dtype in ("float32", "bfloat16"):
        rp = TraceReplayer(None, dtype, max_tokens=640, block_size=8, max_live=1, architecture="Vugotar", model_config=cfg, tensors=tensors)
        for cuts in ((0, n), (0, 2, 560, 561, n)):
            rows = [rp.step({"step": i, "entries": [{"id": "a", "tokens": toks[a:b], "want": list(range(b - a))}], "end": ["a"] if b == n else []})
                    for i, (a, b) in enumerate(zip(cuts, cuts[1:]))]
            within({"r0": np.concatenate(rows)}, {"r0": ref}, dtype, f"cut at {cuts}")


def _model_folder(path, raw, tensors):
    from kvcm_amd.weights.safetensors_io import write_safetensors
    os.makedirs(path)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(raw, f)
    write_safetensors(os.path.join(path, "model.safetensors"), {k: v.to(torch.bfloat16) for k, v in tensors.items()})
    return path


@pytest.mark.parametrize("name", list(cases.CONFIGS))
def test_greedy_generation_through_the_engine(name, tmp_path):
    """The entry point a user calls: model folder -> scheduler -> steps (recorded and replayed, decode steps as graphs) ->
    greedy tokens; against the plain implementation's own greedy continuation."""
    from kvcm_amd import Engine, EngineConfig
    raw = cases.CONFIGS[name]
    cfg, tensors = cases.tensors_for(raw, seed=7 if name in "TU" else 5)
    d = _model_folder(str(tmp_path / "m"), raw, tensors)
    t = cases.as_numpy(tensors)
    prompts = list(cases.requests_for(raw, (9, 30, 1, 17), seed=8).values())
    new = 24
    want, margins = [], []
    for p in prompts:
        toks = list(p)
        for _ in range(new):
            row = plain.forward(raw, t, toks)[-1]
            best = np.sort(row)[-2:]
            margins.append(best[1] - best[0])
            toks.append(int(np.argmax(row)))
        want.append(toks[len(p):])
    assert min(margins) > 1e-3      # no choice is so close that 32-bit rounding could decide it
    for chunk in (0, 8):
        eng = Engine(d, EngineConfig(dtype="float32", block_size=cases.BLOCK_SIZE[name], max_seq_len=128, num_blocks=40,
                                     max_num_seqs=3, max_batched_tokens=64, prefill_chunk=chunk))
        assert eng.recorded is not None          # steps are recorded and replayed, decode steps as graphs: as for the other designs
        got = eng.generate(prompts, new)
        assert got == want, f"prefill_chunk={chunk}"


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_trace_run_program_reads_the_model_folder(dtype, tmp_path):
    raw = cases.CONFIGS["Q"]
    cfg, tensors = cases.tensors_for(raw, seed=9)
    d, out = _model_folder(str(tmp_path / "m"), raw, tensors), str(tmp_path / "out")
    reqs = cases.requests_for(raw, (40, 7, 19, 70), seed=4)
    steps = schedule_mixed(reqs, seed=4, max_live=3)
    p = subprocess.run([os.path.join(ROOT, "bin", "trace_run"), "--model", d, "--dtype", dtype, "--out", out, "--max-tokens", "256"],
                       input="\n".join(json.dumps(s) for s in steps) + "\n", capture_output=True, text=True, timeout=600)
    assert p.returncode == 0, p.stderr[-2000:]
    assert [l for l in p.stdout.split("\n") if l.startswith("done")] == [f"done {s['step']}" for s in steps]
    t = cases.as_numpy(tensors)
    ref = {rid: plain.forward(raw, t, toks) for rid, toks in reqs.items()}
    got = {rid: np.full_like(ref[rid], np.nan, dtype=np.float32) for rid in reqs}
    pos = {rid: 0 for rid in reqs}
    for s in steps:
        rows = np.fromfile(os.path.join(out, f"{s['step']}.f32"), dtype="<f4").reshape(-1, raw["vocab"])
        r = 0
        for e in s["entries"]:
            for w in e["want"]:
                got[e["id"]][pos[e["id"]] + w] = rows[r]
                r += 1
            pos[e["id"]] += len(e["tokens"])
    within(got, ref, dtype, "trace_run")


def test_the_serving_tools_take_the_design(tmp_path):
    """kvmodel writes a random model folder from a configuration file, kvgen generates from it (greedy, against the plain
    implementation on the folder's own tensors), kvbench serves a small workload with random weights of it."""
    cfg_file = str(tmp_path / "p.json")
    with open(cfg_file, "w") as f:
        json.dump(cases.CONFIGS["P"], f)
    d = str(tmp_path / "m")
    tool = lambda name, *args: subprocess.run([sys.executable, os.path.join(ROOT, "bin", name), *args], capture_output=True,
                                              text=True, timeout=300)
    p = tool("kvmodel", "--out", d, "--config-json", cfg_file, "--weights-seed", "3", "--std", "0.15", "--norm-jitter", "0.1")
    assert p.returncode == 0 and "Vugotar" in p.stdout, p.stderr
    prompt = [5, 17, 3, 90, 41, 77, 9]
    p = tool("kvgen", "--model", d, "--dtype", "fp32", "--prompt-ids", ",".join(map(str, prompt)), "--max-new-tokens", "10",
             "--max-seq-len", "64", "--num-blocks", "16")
    assert p.returncode == 0, p.stderr
    t = plain.read_tensors(os.path.join(d, "model.safetensors"))
    toks = list(prompt)
    for _ in range(10):
        toks.append(int(np.argmax(plain.forward(cases.CONFIGS["P"], t, toks)[-1])))
    assert [int(x) for x in p.stdout.split()] == toks[len(prompt):]
    p = tool("kvbench", "--random-weights", "--config-json", cfg_file, "--dtype", "bf16", "--requests", "6", "--prompt-len", "9",
             "--output-len", "5", "--max-seq-len", "64", "--num-blocks", "32", "--warmup", "1")
    assert p.returncode == 0, p.stderr + p.stdout
