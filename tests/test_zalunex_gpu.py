"""The Zalunex decoder in the engine against the plain implementation (tests/plain_zalunex.py): every mechanism alone
through its kernels, then whole models of small odd sizes through the step function, the cache manager, the replayer's
schedules and the engine's own entry point."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

import plain_zalunex as plain
import zalunex_cases as cases
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
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("H", [48, 50, 1030])
def test_embedding_with_a_vector_per_position(H, dtype):
    from kvcm_amd import ops
    rng = np.random.default_rng(H)
    table, pos_table = bf16_grid(rng.normal(size=(9, H))), bf16_grid(rng.normal(size=(40, H)))
    ids, pos = [3, 8, 0, 3, 5], [0, 39, 7, 1, 38]
    out = torch.empty(5, H, device=DEV)
    ops.embed_scaled(i32(ids), dev(table, dtype), out, 1.0, positions=i32(pos), pos_table=dev(pos_table, dtype))
    np.testing.assert_allclose(out.cpu().numpy(), table[ids] + pos_table[pos], atol=1e-6)
    # the embedding's factor does not touch the position's vector; without a table of positions nothing is added
    ops.embed_scaled(i32(ids), dev(table, dtype), out, 0.25, positions=i32(pos), pos_table=dev(pos_table, dtype))
    np.testing.assert_allclose(out.cpu().numpy(), 0.25 * table[ids] + pos_table[pos], atol=1e-6)
    ops.embed_scaled(i32(ids), dev(table, dtype), out, 0.25)
    np.testing.assert_allclose(out.cpu().numpy(), 0.25 * table[ids], atol=1e-6)
    with pytest.raises(ValueError, match="need the positions"):
        ops.embed_scaled(i32(ids), dev(table, dtype), out, 1.0, pos_table=dev(pos_table, dtype))


def test_norms_on_both_sides_with_a_factor_on_what_is_added():
    """x += factor * n(y) * (1 + w_b), then n(x) * (1 + w), in one launch; y as a tensor, as the slices of a split product, and as what
    a joined mixer hands on."""
    from kvcm_amd import ops
    from kvcm_amd.parts.base import BuildContext
    from kvcm_amd.parts.chain_norm_parts import ChainedRMSNorm
    rng = np.random.default_rng(1)
    for T, H in ((5, 48), (3, 321), (2, 4100)):
        x, y, w, wb = rng.normal(size=(T, H)) * 2, rng.normal(size=(T, H)), 0.3 * rng.normal(size=H), 0.3 * rng.normal(size=H)
        parts = rng.normal(size=(3, T, H))
        parts[0] = y - parts[1:].sum(0)
        ctx = BuildContext(torch.float32, torch.device(DEV), H, 16, ops)
        for factor in (1.0, 0.35, -1.2):
            inner = ChainedRMSNorm({"size": H, "eps": 1e-5, "offset": 1.0}, "a.", ctx)
            outer = ChainedRMSNorm({"size": H, "eps": 1e-5, "offset": 1.0, "factor": factor}, "b.", ctx)
            inner.bind({"weight": dev(w)})
            outer.bind({"weight": dev(wb)})
            want = x + factor * plain.offset_norm(y, wb, 1e-5)
            split = lambda: ops.PartialSums(dev(parts), 3, T, H, torch.empty(T, H, device=DEV))
            for value in (dev(y), split(), ops.StreamTerms([(dev(y), 1.0)]), ops.StreamTerms([(split(), 1.0)])):
                xs, out = dev(x), torch.empty(T, H, device=DEV)
                inner.forward(xs, out, add=outer.pending(value))
                np.testing.assert_allclose(xs.cpu().numpy(), want, atol=1e-5 * np.abs(want).max())
                np.testing.assert_allclose(out.cpu().numpy(), plain.offset_norm(want, w, 1e-5), atol=2e-5)
        with pytest.raises(ValueError, match="more than one plain term"):
            outer.pending(ops.StreamTerms([(dev(y), 1.0), (dev(y), 1.0)]))


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
@pytest.mark.parametrize("shape", [dict(nh=4, nkv=2, d=16, dv=16, B=16, W=20), dict(nh=3, nkv=1, d=32, dv=24, B=8, W=33), dict(nh=2, nkv=2, d=10, dv=14, B=8, W=0),
                                   dict(nh=2, nkv=1, d=64, dv=64, B=16, W=1), dict(nh=6, nkv=2, d=128, dv=128, B=32, W=70), dict(nh=4, nkv=1, d=24, dv=16, B=16, W=64),
                                   dict(nh=2, nkv=2, d=64, dv=40, B=16, W=150), dict(nh=1, nkv=1, d=64, dv=130, B=16, W=48)])
def test_window_attention_with_sinks_and_gates_per_head_and_keys_that_stand_out_at_every_edge(shape, dtype):
    """One key is made to dominate the scores of the last row; it is put far away, at page borders, at the first position, just
    inside and just outside the last row's window; decoded rows and runs of rows, through shuffled pages with rubbish in the
    others and with the passed pages given back; every head with a sink and a gate of its own."""
    from kvcm_amd import ops
    s = shape
    nh, nkv, d, dv, B, W = (s[k] for k in ("nh", "nkv", "d", "dv", "B", "W"))
    rng = np.random.default_rng(nh * 100 + d + W)
    n, scale, factor = 230, 0.1, 0.8
    last = n - 1
    sink = np.linspace(-2.0, 4.0, nh)
    spots = {0, B - 1, 2 * B, last - 1, last, 64, 63, 128}
    if W:
        spots |= {last - W, last - W + 1, last - W - 1, last - W + 2}
    pos = np.arange(n)
    for spot in sorted(p for p in spots if 0 <= p <= last):
        k, v, q = rng.normal(size=(n, nkv, d)), rng.normal(size=(n, nkv, dv)), rng.normal(size=(n, nh, d))
        k[spot] *= 4.0
        q[last] = np.repeat(k[spot], nh // nkv, axis=0) * 1.5
        if dtype == torch.bfloat16:
            k, v, q = bf16_grid(k), bf16_grid(v), bf16_grid(q)
        gates = rng.normal(size=(n, nh + 3)) * 2
        want = plain.window_attention(q, k, v, scale, sink, pos, pos, W) * factor * plain.logistic(gates[:, 1:1 + nh])[:, :, None]
        tol = 3e-5 if dtype == torch.float32 else 3e-2
        for first in (last, last - 9, 100, 0):
            passed = max(first + 1 - W, 0) // B if W else 0      # pages wholly before the window of the run's first row
            kc, vc, table = _paged(rng, k, v, B, dtype, passed)
            st = Runs([(first, n - first, 0)])
            tables = i32(table)
            out = torch.full((n - first, nh * dv + 6), 7.0, dtype=dtype, device=DEV)      # a view into wider rows, as a joined layer hands it over
            qd = dev(q[first:].reshape(n - first, -1), dtype)
            rule = dict(sink=dev(sink), out_scale=factor, gate=dev(gates[first:])[:, 1:], gate_heads=True)
            ops.attention_window_pool(qd, out[:, 3:3 + nh * dv], kc, vc, None, None, tables, len(table), st.row_seq, st.ctx_lens, nh, nkv, d, dv, scale,
                                      W, 0, **rule)
            np.testing.assert_allclose(out[:, 3:3 + nh * dv].float().cpu().numpy(), want[first:].reshape(n - first, -1), atol=tol, err_msg=f"key {spot} rows from {first}")
            assert float((out[:, :3].float() - 7.0).abs().max()) == 0.0 and float((out[:, 3 + nh * dv:].float() - 7.0).abs().max()) == 0.0
            if ops.attention_window_pool_tiles_supported(d, dv, dtype, B):
                out2 = torch.empty(n - first, nh * dv + 6, dtype=dtype, device=DEV)
                ops.attention_window_pool_tiles(qd, out2[:, 3:3 + nh * dv], kc, vc, None, None, tables, len(table), st.run_start, st.seq_start, 1, n - first,
                                                nh, nkv, d, dv, scale, W, 0, **rule)
                np.testing.assert_allclose(out2[:, 3:3 + nh * dv].float().cpu().numpy(), want[first:].reshape(n - first, -1), atol=tol,
                                           err_msg=f"tiles: key {spot} rows from {first}")


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_a_sink_far_above_and_far_below_the_scores(dtype):
    """A sink that takes nearly all of the weight, one that takes none, and scores so large that only a running maximum over both
    keeps them in range."""
    from kvcm_amd import ops
    rng = np.random.default_rng(1)
    n, d, dv, B, W = 90, 32, 32, 16, 40
    v = bf16_grid(rng.normal(size=(n, 1, dv)) + 2.0)
    k = np.zeros((n, 1, d))
    k[:, 0, 0] = 1.0
    sink = np.array([8.0, -30.0, 95.0, 0.0])
    for level in (-6.0, 0.0, 90.0):
        q = np.zeros((n, 4, d))
        q[:, :, 0] = level
        want = plain.window_attention(q, k, v, 1.0, sink, np.arange(n), np.arange(n), W)
        kc, vc, table = _paged(rng, k, v, B, dtype, 0)
        st = Runs([(0, n, 0)])
        tol = 2e-5 if dtype == torch.float32 else 2e-2
        out = torch.empty(n, 4 * dv, dtype=dtype, device=DEV)
        ops.attention_window_pool(dev(q.reshape(n, -1), dtype), out, kc, vc, None, None, i32(table), len(table), st.row_seq, st.ctx_lens, 4, 1, d, dv, 1.0, W, 0,
                                  sink=dev(sink))
        np.testing.assert_allclose(out.float().cpu().numpy(), want.reshape(n, -1), atol=tol)
        if dtype == torch.bfloat16:
            ops.attention_window_pool_tiles(dev(q.reshape(n, -1), dtype), out, kc, vc, None, None, i32(table), len(table), st.run_start, st.seq_start, 1, n, 4, 1,
                                            d, dv, 1.0, W, 0, sink=dev(sink))
            np.testing.assert_allclose(out.float().cpu().numpy(), want.reshape(n, -1), atol=tol)
        assert np.abs(want[:, 2]).max() < (0.5 if level < 90 else 3.0) and np.abs(want[60, 1]).max() > 1.0


DECAYS = (0.9, 0.0, 1.0, 0.5)


@pytest.mark.parametrize("silu", [False, True])
@pytest.mark.parametrize("shape", [(4, 12, 20), (3, 32, 8), (2, 64, 40), (1, 5, 3), (2, 1, 1), (4, 96, 17), (2, 130, 33), (1, 256, 70), (2, 48, 130), (3, 64, 64), (2, 128, 128)])
def test_states_with_a_constant_decay_over_runs_cut_at_random(shape, silu):
    """Two sequences of unequal length, their runs interleaved in steps and cut at random, slots that held rubbish: walked row by
    row, walked in pieces, in matrix form with every run one piece, and in matrix form in pieces of 64 rows; a step may mix forms."""
    from kvcm_amd import ops
    heads, dk, dv = shape
    rng = np.random.default_rng(sum(shape))
    lens, decay = (230, 120), DECAYS[:heads]
    data = [[rng.normal(size=(n, heads, c)) for c in (dk, dk, dv)] for n in lens]
    act = plain.silu if silu else (lambda x: x)
    want = [plain.decayed_state(*(act(x) for x in d), decay) for d in data]
    top = max(np.abs(w).max() for w in want)
    for form in ("walk", "walk in pieces", "matrix", "matrix in pieces", "any"):
        state = torch.full((4, heads, dk, dv), float("nan"), device=DEV)
        done, got = [0, 0], [np.zeros((n, heads * dv)) for n in lens]
        while any(d < n for d, n in zip(done, lens)):
            runs, take = [], []
            for s in rng.permutation(2):
                n = min(int(rng.choice([1, 2, 9, 30, 64, 65, 150])), lens[s] - done[s])
                if n:
                    runs.append((done[s], n, (3, 1)[s]))
                    take.append((s, done[s], n))
                    done[s] += n
            st = Runs(runs)
            q, k, v = (dev(np.concatenate([data[s][i][p:p + n].reshape(n, -1) for s, p, n in take])) for i in range(3))
            o = torch.full((st.rows, heads * dv), float("nan"), device=DEV)
            how = form if form != "any" else str(rng.choice(["walk", "matrix", "matrix in pieces"]))
            nan = lambda count: torch.full((count,), float("nan"), device=DEV)
            if how.startswith("walk"):
                carry = nan(ops.gated_state_carry_floats(st.rows, st.seqs, heads, dk, dv, False, 8)) if how != "walk" else None
                ops.gated_state(q, k, v, None, None, None, o, state, st, heads, heads, dk, dv, decay=dev(decay), silu_in=silu, carry=carry, piece=8)
            else:
                piece = 64 if how != "matrix" else 256
                carry = nan(ops.lightning_carry_floats(st.rows, st.seqs, heads, dk, dv, piece)) if how != "matrix" else None
                ops.lightning(q, k, v, ops.lightning_powers(decay, piece, DEV), o, state, st, heads, dk, dv, silu_in=silu, carry=carry, piece=piece)
            r = 0
            for s, p, n in take:
                got[s][p:p + n] = o[r:r + n].cpu().numpy()
                r += n
        for s in range(2):
            np.testing.assert_allclose(got[s], want[s].reshape(lens[s], -1), atol=1e-5 * top, err_msg=f"sequence {s}, {form}")
        assert torch.isnan(state[[0, 2]]).all() and not torch.isnan(state[[1, 3]]).any()


def test_rows_of_a_view_and_sequences_without_a_slot():
    """The projections as columns of wider rows at places that are no multiple of four, and a padding sequence: its outputs are zero,
    nothing of it is kept."""
    from kvcm_amd import ops
    rng = np.random.default_rng(4)
    heads, dk, dv, n = 2, 20, 12, 70
    wide = rng.normal(size=(2 * n, 3 + heads * (2 * dk + dv) + 2))
    cols = [wide[:, 3:3 + heads * dk], wide[:, 3 + heads * dk:3 + 2 * heads * dk], wide[:, 3 + 2 * heads * dk:3 + heads * (2 * dk + dv)]]
    want = plain.decayed_state(*(c[:n].reshape(n, heads, -1) for c in cols), (0.9, 0.99)).reshape(n, -1)
    st = Runs([(0, n, 1), (0, n, -1)])
    w = dev(wide)
    q, k, v = w[:, 3:], w[:, 3 + heads * dk:], w[:, 3 + 2 * heads * dk:]
    state = torch.full((2, heads, dk, dv), float("nan"), device=DEV)
    for piece in (64, 128):
        o = torch.full((2 * n, heads * dv), float("nan"), device=DEV)
        carry = torch.full((ops.lightning_carry_floats(2 * n, 2, heads, dk, dv, piece),), float("nan"), device=DEV)
        ops.lightning(q, k, v, ops.lightning_powers((0.9, 0.99), piece, DEV), o, state, st, heads, dk, dv, carry=carry, piece=piece)
        np.testing.assert_allclose(o[:n].cpu().numpy(), want, atol=1e-5 * np.abs(want).max())
        assert not o[n:].any() and torch.isnan(state[0]).all()
    with pytest.raises(ValueError, match="longer than a piece"):
        ops.lightning(q, k, v, ops.lightning_powers((0.9, 0.99), 64, DEV), o, state, st, heads, dk, dv, piece=64)


def test_a_token_written_hundreds_of_rows_ago_comes_back_through_every_piece():
    """The state as a lookup: one key, orthogonal to all others, is written at row 3 and asked for at the last of 700 rows, across
    pieces of the kernels' own size, from a slot and from nothing."""
    from kvcm_amd import ops
    rng = np.random.default_rng(2)
    T, heads, dk, dv, decay = 700, 2, 32, 24, (1.0, 0.999)
    q, k, v = (rng.normal(size=(T, heads, c)) for c in (dk, dk, dv))
    k[:, :, 0] = 0.0
    k[3], q[-1] = 0.0, 0.0
    k[3, :, 0] = q[-1, :, 0] = 1.0
    want = plain.decayed_state(q, k, v, decay)
    np.testing.assert_allclose(want[-1], v[3] * np.array([[1.0], [0.999 ** 696]]), atol=1e-9)
    powers = ops.lightning_powers(decay, ops.lightning_piece(dk), DEV)
    for cut in (0, 2, 150):
        state = torch.full((2, heads, dk, dv), float("nan"), device=DEV)
        rows = []
        for lo, hi in ((0, cut), (cut, T)):
            if lo == hi:
                continue
            st = Runs([(lo, hi - lo, 1)])
            o = torch.empty(hi - lo, heads * dv, device=DEV)
            carry = torch.full((ops.lightning_carry_floats(hi - lo, 1, heads, dk, dv),), float("nan"), device=DEV)
            part = lambda x: dev(x[lo:hi].reshape(hi - lo, -1))
            ops.lightning(part(q), part(k), part(v), powers, o, state, st, heads, dk, dv, carry=carry)
            rows.append(o.cpu().numpy())
        got = np.concatenate(rows)
        np.testing.assert_allclose(got, want.reshape(T, -1), atol=2e-5 * np.abs(want).max(), err_msg=f"cut at {cut}")
        np.testing.assert_allclose(got[-1], want[-1].reshape(-1), atol=2e-5)


def test_gates_norms_activations_and_routing_alone():
    """The norm over all heads before its gate; the gate with limits, on its own and in the product's epilogue, with values on both
    sides of every limit; the exact gelu; sigmoid scores as weights."""
    from kvcm_amd import ops
    rng = np.random.default_rng(6)
    for T, size in ((5, 48), (2, 50), (3, 1400), (2, 3000), (2, 5000)):
        y, z, w = rng.normal(size=(T, size)), rng.normal(size=(T, size + 4)) * 2, 1 + 0.2 * rng.normal(size=size)
        want = plain.rms(y, 1e-5) * w * plain.logistic(z[:, :size])
        for dt, tol in ((torch.float32, 1e-5), (torch.bfloat16, 2.0 ** -7)):
            out = torch.zeros(T, size + 3, dtype=dt, device=DEV)
            ops.group_norm_gate(dev(y), dev(z), dev(w), out[:, 1:1 + size], 1, size, 1e-5, after=True)
            np.testing.assert_allclose(out[:, 1:1 + size].float().cpu().numpy(), want, atol=tol * np.abs(want).max())
            assert not out[:, 0].any() and not out[:, 1 + size:].any()
    T, I = 7, 37
    for limit in (0.4, 1.0, 6.0):
        gu = rng.normal(size=(T, 2 * I + 3)) * 2
        gu[0, :4], gu[0, I:I + 4] = (limit, 30.0, -30.0, limit * 1.01), (-30.0, limit, 30.0, -limit * 1.01)
        want = plain.clamped_gate(gu[:, :I], gu[:, I:2 * I], limit)
        for dt, tol in ((torch.float32, 2e-6), (torch.bfloat16, 2.0 ** -8)):
            out = torch.empty(T, I + 5, dtype=dt, device=DEV)
            ops.gated_act(dev(gu), out[:, 2:2 + I], "clamped", limit=limit)
            np.testing.assert_allclose(out[:, 2:2 + I].float().cpu().numpy(), want, atol=tol * max(1.0, np.abs(want).max()))
    with pytest.raises(Exception, match="positive limit"):
        ops.gated_act(dev(gu), out[:, :I], "clamped")
    for M, K, I, limit in ((1, 256, 5120, 0.9), (8, 128, 5632, 2.0), (40, 64, 5120, 0.5), (3, 64, 2568, 1.1)):
        x, wm = bf16_grid(rng.normal(size=(M, K))), bf16_grid(rng.normal(size=(2 * I, K)) * 2 * K ** -0.5)
        act = torch.empty(M, I, dtype=torch.bfloat16, device=DEV)
        assert ops.gemm_swiglu(dev(x, torch.bfloat16), dev(wm, torch.bfloat16), act, limit=limit)
        g = x @ wm.T
        want = plain.clamped_gate(g[:, :I], g[:, I:], limit)
        np.testing.assert_allclose(act.float().cpu().numpy(), want, atol=2.0 ** -8 * max(1.0, np.abs(want).max()), err_msg=f"{M} x {K} x {I}")
    z = np.linspace(-9.0, 9.0, 5 * 64).reshape(5, 64)
    for dt, tol in ((torch.float32, 2e-6), (torch.bfloat16, 2.0 ** -8)):
        out = torch.empty(5, 64, dtype=dt, device=DEV)
        ops.act_rows(dev(z), out, "gelu")
        np.testing.assert_allclose(out.float().cpu().numpy(), plain.gelu(z), atol=tol * 9)
    for E, top, factor in ((8, 4, 2.5), (5, 1, 0.3), (1, 1, 1.0), (70, 6, 1.7)):
        z = rng.normal(size=(9, E)) * 2
        want_c, want_w = plain.choose_experts(z, top)
        chosen, weight = torch.empty(9, top, dtype=torch.int32, device=DEV), torch.empty(9, top, device=DEV)
        ops.moe_route(dev(z), E, top, chosen, weight, sigmoid=True, factor=factor)
        assert chosen.cpu().numpy().tolist() == want_c.tolist()
        np.testing.assert_allclose(weight.cpu().numpy(), want_w * factor, atol=3e-6 * factor)


@pytest.mark.parametrize("gated", [False, True])
@pytest.mark.parametrize("shape", [(3, 4, 2, 24, 20, 24), (70, 5, 3, 64, 32, 64), (200, 3, 1, 136, 144, 136), (33, 2, 2, 40, 8, 40), (260, 6, 2, 64, 200, 64), (18, 1, 1, 48, 50, 48)])
def test_experts_whose_weight_acts_on_what_they_read(shape, gated):
    """gelu (and gated) experts, a row at a time and grouped by expert; weights far from one, so that the two sides differ."""
    from kvcm_amd import ops
    from kvcm_amd.parts.routed_parts import interleave_gate_up
    T, E, top, K, F, H = shape
    if gated:
        F = -(-F // 16) * 16
    rng = np.random.default_rng(T + E + F)
    h, up, gate = bf16_grid(rng.normal(size=(T, K))), bf16_grid(rng.normal(size=(E, F, K)) * 1.5 * K ** -0.5), bf16_grid(rng.normal(size=(E, F, K)) * 1.5 * K ** -0.5)
    down = bf16_grid(rng.normal(size=(E, H, F)) * F ** -0.5)
    chosen = np.stack([rng.permutation(E)[:top] for _ in range(T)])
    weight = rng.uniform(0.1, 2.5, size=(T, top))
    add = rng.normal(size=(T, H))

    def expert(x, e):
        return (plain.silu(gate[e] @ x) * (up[e] @ x) if gated else plain.gelu(up[e] @ x)) @ down[e].T

    want_in = np.stack([add[t] + sum(expert(a * h[t], e) for e, a in zip(chosen[t], weight[t])) for t in range(T)])
    want_out = np.stack([add[t] + sum(a * expert(h[t], e) for e, a in zip(chosen[t], weight[t])) for t in range(T)])
    assert np.abs(want_in - want_out).max() > 0.1
    for dt, tol in ((torch.float32, 2e-5), (torch.bfloat16, 3e-2)):
        u, d = dev(up, dt), dev(down, dt)
        if gated:
            u = interleave_gate_up(dev(gate, dt), u)
        c, w = i32(chosen.reshape(-1)).view(T, top), dev(weight)
        how = dict(gated=gated, add=dev(add), **({} if gated else {"activation": "gelu"}))
        for weigh_input, want in ((True, want_in), (False, want_out)):
            act, out = torch.empty(T * top, F, dtype=dt, device=DEV), torch.empty(T, H, device=DEV)
            ops.moe_rows(dev(h, dt), u, d, c, w, act, out, weigh_input=weigh_input, **how)
            np.testing.assert_allclose(out.cpu().numpy(), want, atol=tol * max(1.0, np.abs(want).max()))
            if ops.moe_grouped_supported(K, F, E, dt):
                order = torch.empty(T * top, dtype=torch.int32, device=DEV)
                tiles = torch.empty(ops.moe_grouped_tiles(T * top, E), dtype=torch.int32, device=DEV)
                y, out2 = torch.empty(T * top, H, device=DEV), torch.full((T, H), float("nan"), device=DEV)
                ops.moe_grouped(dev(h, dt), u, d, c, w, order, tiles, act, y, out2, weigh_input=weigh_input, **how)
                np.testing.assert_allclose(out2.cpu().numpy(), want, atol=tol * max(1.0, np.abs(want).max()))
    with pytest.raises(ValueError, match="unknown activation"):
        ops.moe_rows(dev(h), dev(up), dev(down), c, w, torch.empty(T * top, F, device=DEV), out, activation="silu")


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


@pytest.mark.parametrize("rows", [1, 21, 150])
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_sublayers_run_on_their_own_and_joined(dtype, rows):
    """The lightning half by itself, the feed-forwards by themselves, and the two halves of a mixer joined with their factors, each
    against its plain function (the attention half needs pages: here it stands in as a second lightning part)."""
    from kvcm_amd import ops
    from kvcm_amd.parts.base import BuildContext, PartSpec
    from kvcm_amd.parts.joined_parts import JoinedSublayers
    from kvcm_amd.registry import FEED_FORWARDS, MIXERS
    rng = np.random.default_rng(9)
    H, T, eps = 40, rows, 1e-5
    h = bf16_grid(rng.normal(size=(T, H)))
    a = {"heads": 3, "dim": 12, "vdim": 10, "decay": (0.9, 0.99, 0.4), "eps": eps}
    b = {"heads": 2, "dim": 8, "vdim": 20, "decay": (0.7, 1.0), "eps": eps}
    specs = {"a": ("mixer", PartSpec("lightning_attention", a, "a.")), "b": ("mixer", PartSpec("lightning_attention", b, "b.")),
             "dense": ("ffn", PartSpec("gated_mlp", {"intermediate_size": 24, "activation": "clamped", "limit": 0.7, "partial_out": True}, "f.")),
             "experts": ("ffn", PartSpec("routed_experts", {"experts": 5, "top": 5, "ff": 12, "routing": "sigmoid", "activation": "gelu", "weigh": "input"}, "e."))}
    context = lambda: BuildContext(dtype, torch.device(DEV), H, 16, ops)
    tensors = {}

    def bind(part):
        for p in [*part.sub_parts(), part]:
            bound = {}
            for ps in p.param_specs():
                for name, shape in ps.sources:
                    if name not in tensors:
                        x = rng.normal(size=shape) * (shape[-1] ** -0.5 if len(shape) == 2 else 0.3) + (1.0 if ps.role == "vector" else 0.0)
                        tensors[name] = bf16_grid(x)
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
        x = torch.zeros(T, H, device=DEV)
        ops.stream_terms(x, eps, add=ops.StreamTerms.of(value))
        return x.cpu().numpy()

    got = {}
    for name, (registry, spec) in specs.items():
        part = bind((MIXERS if registry == "mixer" else FEED_FORWARDS).get(spec.kind)(spec.params, spec.prefix, context()))
        states(part)
        got[name] = total(part.forward(Alone([(0, T, 1)], ops, dtype), dev(h, dtype)))
    t = tensors
    want = {"a": plain.lightning(h, t, "a.", a, eps), "b": plain.lightning(h, t, "b.", b, eps), "dense": plain.dense_ff(h, t, "f.", 0.7),
            "experts": plain.mixture(h, t, "e.", {"router": {"top": 5}})}
    tol = 2e-5 if dtype == torch.float32 else 4e-2
    for name in specs:
        np.testing.assert_allclose(got[name], want[name], atol=tol * max(1.0, np.abs(want[name]).max()), err_msg=name)
    listed = tuple((n, "mixer", PartSpec("lightning_attention", {**p, "out_factor": f}, n + ".")) for n, p, f in (("a", a, 0.6), ("b", b, -1.4)))
    part = bind(JoinedSublayers({"members": listed}, "l.", context()))
    for member in part.members:
        states(member)
    joined = 0.6 * want["a"] - 1.4 * want["b"]
    np.testing.assert_allclose(total(part.forward(Alone([(0, T, 1)], ops, dtype), dev(h, dtype))), joined, atol=tol * max(1.0, np.abs(joined).max()))


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
                               architecture="Zalunex", model_config=cfg, tensors=tensors)
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
            out = original(step, x, pending)      # what the layer adds is still pending: normed and added to a copy here
            ops, stream = model.ctx.ops, x.clone()
            ops.rmsnorm_chain(stream, raw["norm"]["eps"], pending=out)
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


@pytest.mark.parametrize("case", [("P", "float32"), ("Q", "bfloat16"), ("R", "bfloat16"), ("S", "float32"), ("U", "bfloat16")])
def test_steps_replayed_from_recorded_launch_lists(models, case):
    """Every part says it is capturable: a step's shape is recorded once as a list of launches and replayed with only the
    step's metadata changed; padding rows and padding sequences must leave the pages alone."""
    from kvcm_amd.engine.replay import TraceReplayer
    _, reqs, ref, raw, _ = models(*case)
    cfg, tensors = cases.tensors_for(raw, seed=len(case[0]) + sum(map(ord, case[0])))
    rp = TraceReplayer(None, case[1], max_tokens=tokens_needed(reqs, 3), block_size=cases.BLOCK_SIZE[case[0]], max_live=3,
                       architecture="Zalunex", model_config=cfg, tensors=tensors, use_programs=True)
    assert rp.programs is not None
    for steps in (schedule_mixed(reqs, seed=5, max_live=3), schedule_tail_singly(reqs, tail=20)):
        within(replay(rp, steps, reqs), ref, case[1], str(case))
    assert rp.steps_replayed > 50


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["P", "Q", "R", "S", "V"])
def test_long_decoding_far_beyond_every_window(name, dtype):
    """300 tokens one by one: every window passes over decoded tokens, states carry on; passed pages are given back, an attention
    without a window keeps everything."""
    from kvcm_amd.engine.replay import TraceReplayer
    raw = cases.CONFIGS[name] if dtype == "float32" else cases.with_every_expert_chosen(cases.CONFIGS[name])
    cfg, tensors = cases.tensors_for(raw, seed=1 + ord(name))
    n = 300
    toks = cases.requests_for(raw, (n,), seed=11)["r0"]
    ref = {"r0": plain.forward(raw, cases.as_numpy(tensors), toks)}
    steps = [{"step": 0, "entries": [{"id": "r0", "tokens": toks[:4], "want": [0, 1, 2, 3]}], "end": []}]
    steps += [{"step": i, "entries": [{"id": "r0", "tokens": [toks[i]], "want": [0]}], "end": []} for i in range(4, n)]
    rp = TraceReplayer(None, dtype, max_tokens=320, block_size=cases.BLOCK_SIZE[name], max_live=2, architecture="Zalunex",
                       model_config=cfg, tensors=tensors)
    within(replay(rp, steps, {"r0": toks}), ref, dtype, name)
    B = cases.BLOCK_SIZE[name]
    tables = rp.tables()["r0"]
    for g, spec in enumerate(rp.core.groups):
        if spec.kind == "state":
            continue
        first_needed = max(n + 1 - spec.window, 0) // B if spec.window else 0      # of the next token's window
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
    """Positions 0, 1, 2 alone and one by one: windows, sinks without keys beside them, learned positions and states at their start."""
    for name in cases.CONFIGS:
        rp, _, _, raw, t = models(name, "float32")
        toks = cases.requests_for(raw, (3,), seed=31)["r0"]
        ref = plain.forward(raw, t, toks)
        rows = [rp.step({"step": i, "entries": [{"id": "f", "tokens": [toks[i]], "want": [0]}], "end": ["f"] if i == 2 else []})[0] for i in range(3)]
        np.testing.assert_allclose(np.stack(rows), ref, atol=3e-5 * np.abs(ref).max(), err_msg=name)


def test_a_prompt_long_enough_to_be_walked_in_pieces():
    """A prompt of several of the recurrence's pieces in one step, and cut so that one portion takes the pieces, one the matrix form
    alone and one the walk."""
    from kvcm_amd.engine.replay import TraceReplayer
    raw = cases.CONFIGS["U"]
    cfg, tensors = cases.tensors_for(raw, seed=14)
    n = 620
    toks = cases.requests_for(raw, (n,), seed=12)["r0"]
    ref = plain.forward(raw, cases.as_numpy(tensors), toks)
    for dtype in ("float32", "bfloat16"):
        rp = TraceReplayer(None, dtype, max_tokens=640, block_size=8, max_live=1, architecture="Zalunex", model_config=cfg, tensors=tensors)
        for cuts in ((0, n), (0, 2, 560, 561, 581, n)):
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
    cfg, tensors = cases.tensors_for(raw, seed=5)
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
    assert p.returncode == 0 and "Zalunex" in p.stdout, p.stderr
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


def test_a_sequence_ends_where_the_learned_positions_do(tmp_path):
    """A request that would run past the last learned position stops there, with every token before it right."""
    from kvcm_amd import Engine, EngineConfig
    raw = dict(cases.CONFIGS["V"], max_positions=40)
    cfg, tensors = cases.tensors_for(raw, seed=6)
    d = _model_folder(str(tmp_path / "m"), raw, tensors)
    t = cases.as_numpy(tensors)
    prompt = cases.requests_for(raw, (30,), seed=2)["r0"]
    for beyond in (False, True):
        eng = Engine(d, EngineConfig(dtype="float32", block_size=16, max_seq_len=128, num_blocks=20, max_num_seqs=2, max_batched_tokens=64,
                                     beyond_max_position=beyond))
        got = eng.generate([prompt], 24)[0]
        toks = list(prompt)
        while len(toks) < 40:
            toks.append(int(np.argmax(plain.forward(raw, t, toks)[-1])))
        assert got[:10] == toks[30:40] and len(got) <= 11
