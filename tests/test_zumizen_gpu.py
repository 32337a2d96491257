"""Zumizen on the device: each mechanism's kernels against the plain implementation, then whole models under every
way of cutting requests into steps, and generation through the entry points."""
from __future__ import annotations

import json
import os
import subprocess
import sys
from types import SimpleNamespace

import numpy as np
import pytest
import torch

import helpers
from plain import zumizen as pz
from zumizen_cases import CASES, folder_of, rounded

pytestmark = pytest.mark.gpu
F64 = torch.float64
DEV = "cuda:0"


def _dev(t, dtype=torch.float32):
    return t.to(dtype).to(DEV).contiguous()


def _i32(values):
    return torch.tensor(list(values), dtype=torch.int32, device=DEV)


def _step_ctx(rows, slots, tuned=True):
    """The tables of a step whose requests bring ``rows`` = [(request, first position, end position)], single tokens first."""
    lens = [b - a for _, a, b in rows]
    starts = np.cumsum([0] + lens)[:-1]
    tok_seq = [s for s, n in enumerate(lens) for _ in range(n)]
    from glassbox_amd.engine.context import Workspace
    return SimpleNamespace(q_start=_i32(starts), q_len=_i32(lens), pos0=_i32(a for _, a, _ in rows), tok_seq=_i32(tok_seq),
                           state_slots=_i32(slots[r] for r, _, _ in rows), num_seqs=len(rows), tuned=tuned,
                           host={"max_q_len": max(lens), "n_decode": sum(1 for n in lens if n == 1)},
                           buffer=Workspace(torch.device(DEV)).buffer)


# ------------------------------------------------------------------------------------------ small kernels
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_a_sublayers_rows_biased_normed_with_a_weight_a_column_and_added(dtype):
    from glassbox_amd import ops
    torch.manual_seed(4)
    for n, d, slices in ((5, 64, 1), (70, 50, 1), (3, 7, 1), (600, 320, 3), (9, 4096, 2)):
        x, pieces = torch.randn(n, d, dtype=F64), torch.randn(slices, n, d, dtype=F64)
        w, b = torch.randn(d, dtype=F64), torch.randn(d, dtype=F64)
        for bias in (b, None):
            y = pieces.float().to(F64).sum(0) + (0 if bias is None else bias.float().to(F64))
            want = x.float().to(F64) + pz.unit_rms(y, 1e-3) * w.float().to(F64)
            res, rows = _dev(x), torch.empty(n, d, dtype=dtype, device=DEV)
            ops.norm_add(res, _dev(pieces if slices > 1 else pieces[0]), _dev(w), 1e-3, rows, slices=slices,
                         bias=None if bias is None else _dev(bias), conv=(None, None))
            assert (res.cpu().to(F64) - want).abs().max() < 3e-6 * float(want.abs().max())
            assert torch.equal(rows, res.to(dtype))


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_bounded_logits_and_the_scaled_embedding_beside_the_pairs(dtype):
    from glassbox_amd import ops
    torch.manual_seed(1)
    x = torch.randn(7, 301) * 40
    got = x.to(DEV)
    ops.cap_rows(got, 15.0, 0.5)
    assert (got.cpu() - 15.0 * torch.tanh(x.double() * 0.5 / 15.0)).abs().max() < 1e-5
    table, pairs = torch.randn(11, 20).to(dtype), torch.randn(8, 20).to(dtype)
    toks = [3, 9, 9, 1, 0, 10]
    w = {"embed": table.to(F64), "bigram": pairs.to(F64)}
    want = pz.embed({"embedding": {"scale": 3.5, "bigram": {"buckets": 7, "mul_prev": 5, "mul_cur": 3}}}, w, toks)
    prev = torch.full((3, 1), 99, dtype=torch.int32, device=DEV)
    out = []
    for a, b in ((0, 2), (2, 3), (3, 6)):
        ctx = _step_ctx([(0, a, b)], {0: 2})
        ctx.token_ids = _i32(toks[a:b])
        rows = torch.empty(b - a, 20, device=DEV)
        ops.embed_pairs(_dev(table, dtype), _dev(pairs, dtype), ctx, rows, 7, 5, 3, prev, 3.5)
        out.append(rows.cpu().to(F64))
    assert (torch.cat(out) - want).abs().max() < 1e-5


# ------------------------------------------------------------------------------------------ experts
def _expert_part(d, E, top, ff, dtype, seed):
    from glassbox_amd.parts.moe import RoutedExperts
    g = torch.Generator().manual_seed(seed)
    r = lambda *s: (torch.randn(*s, generator=g, dtype=F64) * s[-1] ** -0.5).to(dtype).to(F64)
    w = {f"m.e{e}.{n}": r(*s) for e in range(E) for n, s in (("gate", (ff, d)), ("up", (ff, d)), ("down", (d, ff)))}
    w["m.router"] = (r(E, d) * 3).to(dtype).to(F64)
    part = RoutedExperts(d, E, top, ff, correction=False, scoring="sigmoid", renorm=False, weigh_in=True)
    part.load({n[2:]: _dev(t, dtype) for n, t in w.items()})
    return part, w


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("d, E, top, ff, n", [(64, 6, 1, 24, 9), (50, 5, 3, 30, 70), (64, 70, 2, 16, 33), (128, 8, 2, 64, 500),
                                              (128, 4, 1, 128, 2600), (64, 3, 3, 16, 65), (96, 40, 3, 8, 300)])
def test_experts_whose_weights_multiply_their_input(dtype, d, E, top, ff, n):
    """Few rows (every expert on every token), many (an expert on its own tokens, by tiles of 64, 128 and 256 rows), routers
    in one kernel and in two; a token whose choice hangs on less than rounding is left out."""
    from glassbox_amd.engine.context import Workspace
    part, w = _expert_part(d, E, top, ff, dtype, seed=E * n)
    h = torch.randn(n, d, dtype=F64, generator=torch.Generator().manual_seed(n)).to(dtype).to(F64)
    margins = []
    want = pz.experts(w, "m.", {"router": {"experts": E, "top": top}}, h, margins=margins)
    clear = margins[0] > 1e-4
    assert clear.double().mean() > 0.95
    for tuned in (True, False):
        ctx = SimpleNamespace(dtype=dtype, tuned=tuned, buffer=Workspace(torch.device(DEV)).buffer)
        y = torch.full((n, d), 7.0, device=DEV)
        made, slices = part.forward(ctx, _dev(h, dtype), y, store=True) or (y, 1)
        got = made.view(-1)[:slices * n * d].view(slices, n, d).sum(0).cpu().to(F64)
        tol = 2e-5 if dtype == torch.float32 else 2e-2
        assert ((got - want)[clear]).abs().max() < tol * float(want.abs().max()), (tuned, part.routed(ctx, n))
    if dtype == torch.bfloat16 and n >= 300 and top < E:
        assert part.routed(ctx, n)


# ------------------------------------------------------------------------------------------ attention
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("H, G, dk, dv, run", [(4, 2, 32, 32, 24), (3, 3, 64, 64, 200), (8, 1, 16, 48, 7), (2, 2, 136, 136, 64),
                                               (3, 1, 40, 24, 0), (4, 4, 96, 96, 0), (6, 3, 128, 128, 50)])
def test_attention_with_a_distance_bias_and_a_sink_at_the_edges_of_runs(dtype, H, G, dk, dv, run):
    """One request of 700 tokens.  Queries are built so that the first key of their own run, the last key of the run before,
    a key far back inside the run and one far back outside it would each take most of the softmax if it were visible, far
    enough above what their distance costs them.  The plain kernel whole, token by token with a workgroup a chunk of
    keys, and the matrix-core kernels for portions and single tokens, against the plain functions."""
    from glassbox_amd import ops
    from glassbox_amd.engine.context import Workspace
    from glassbox_amd.parts.attention import cache_head_cols, paged_attention
    T, P, scale = 700, 16, 0.4
    hc, group, span = cache_head_cols(dk, dv), H // G, run or T
    g = torch.Generator().manual_seed(H * dk + run)
    f = lambda t: t.to(dtype).to(F64)
    q = torch.randn(T, H, hc, generator=g, dtype=F64) * 0.3
    k = torch.randn(T, G, hc, generator=g, dtype=F64) * 0.3
    v = torch.randn(T, G, hc, generator=g, dtype=F64)
    q[..., dk:], k[..., dk:], v[..., dv:] = 0.0, 0.0, 0.0
    k, v = f(k), f(v)
    slopes = pz.slopes(H)
    for i in range(40, T, 7):
        start = i - i % span
        target = [start, start - 1, max(start, i - 150), i - 300, i - 1][(i // 7) % 5]
        if target >= 0:
            for h in range(H):
                key = k[target, h // group]
                q[i, h] += (6.0 + float(slopes[h]) * (i - target)) * key / (scale * float((key ** 2).sum()))
    q = f(q)
    s = pz.biased_scores(q, k, scale)
    p = pz.softmax_plus_one(s, pz.visible(T, run))
    want = torch.stack([p[h] @ v[:, h // group] for h in range(H)], 1).reshape(T, H * hc)
    order = np.random.RandomState(1).permutation(-(-T // P) + 3)[:-(-T // P)].tolist()
    slots = [order[t // P] * P + t % P for t in range(T)]
    pages = -(-T // P) + 3
    k_pages = torch.full(ops.key_pages_shape(pages, G, P, hc), 77.0, dtype=dtype, device=DEV)
    v_pages = torch.full((pages, G, hc, P), -55.0, dtype=dtype, device=DEV)
    heads = _dev(torch.cat([q.reshape(T, -1), k.reshape(T, -1), v.reshape(T, -1)], 1), dtype)
    ops.rope_store(heads, None, None, _i32(slots), k_pages, v_pages, H, G, hc, rotate=False)
    table, sinks, sl = _i32(order).view(1, -1), torch.zeros(H, device=DEV), _dev(slopes)
    limit = (3e-5 if dtype == torch.float32 else 3e-2) * max(1.0, float(want.abs().max()))
    out = torch.empty(T, H * hc, dtype=dtype, device=DEV)
    for grouped in (False, True):
        out.fill_(9.0)
        ops.attention_plain(heads[:, :H * hc], out, _i32(range(T)), _i32([0] * T), table, k_pages, v_pages, H, scale, 0,
                            grouped=grouped, chunk=run, sinks=sinks, slopes=sl)
        assert (out.cpu().to(F64) - want).abs().max() < limit, ("plain kernel, whole", grouped)
    rows = list(range(T - 9, T))
    floats = ops.attention_plain_split_floats(len(rows), H, hc, P, T)
    split = torch.empty(len(rows), H * hc, dtype=dtype, device=DEV)
    ops.attention_plain(heads[rows, :H * hc], split, _i32(rows), _i32([0] * len(rows)), table, k_pages, v_pages, H, scale, 0,
                        workspace=torch.empty(floats, device=DEV), max_context=T, chunk=run, sinks=sinks, slopes=sl)
    assert torch.equal(split, out[rows])
    if dtype != torch.bfloat16 or not ops.tuned_attention_supports(k_pages, H, 0, 0):
        return
    cache = SimpleNamespace(k_pages=k_pages, v_pages=v_pages, group=0)
    ws = Workspace(torch.device(DEV))
    edge = run or 350
    steps = [[[t] for t in (T - 1, edge, edge - 1, min(2 * edge, T) - 1, 0, 300)], [list(range(311))], [[311, 312]], [list(range(313, T))],
             [[T - 1], list(range(100, 430))], [[5], [T - 2], list(range(edge - 1, edge + 40)), [3, 4]]]
    for rows in steps:   # single tokens first, then portions (each as a request of its own)
        flat = [t for r in rows for t in r]
        lens = [len(r) for r in rows]
        ctx = SimpleNamespace(dtype=dtype, tuned=True, tables=[table.expand(len(rows), -1).contiguous()], positions=_i32(flat),
                              tok_seq=_i32(i for i, n in enumerate(lens) for _ in range(n)), q_start=_i32(np.cumsum([0] + lens)[:-1]),
                              q_len=_i32(lens), pos0=_i32(r[0] for r in rows), num_seqs=len(rows), buffer=ws.buffer,
                              host={"n_decode": sum(1 for n in lens if n == 1), "max_q_len": max(lens), "max_context": max(flat) + 1})
        wide = torch.full((len(flat), H * hc + 24), 9.0, dtype=dtype, device=DEV)      # the result as columns of wider rows
        paged_attention(ctx, heads[flat, :H * hc].contiguous(), wide[:, 8:8 + H * hc], cache, H, scale, 0, 0, run, 0.0, sinks, sl)
        got = wide[:, 8:8 + H * hc].cpu().to(F64)
        assert (got - want[flat]).abs().max() < limit, lens
        assert torch.all(wide[:, :8] == 9.0) and torch.all(wide[:, 8 + H * hc:] == 9.0)


# ------------------------------------------------------------------------------------------ the delta rule
DELTA_CASES = [   # H, G, dk, dv, taps, a decay a channel
    (4, 2, 16, 24, 3, False), (2, 2, 32, 16, 4, True), (3, 1, 64, 64, 1, True), (3, 3, 10, 5, 2, False), (2, 1, 6, 9, 3, True),
    (2, 2, 96, 144, 5, True), (1, 1, 128, 32, 8, False), (2, 1, 160, 20, 4, True), (2, 2, 200, 300, 4, False), (1, 1, 128, 256, 2, True)]


def _delta_inputs(lens, H, G, dk, dv, taps, channel, dtype, seed, rate=None):
    """Projections of requests of these lengths and the constants, with what the plain functions make of them: decays between
    almost none and almost all a token."""
    g = torch.Generator().manual_seed(seed)
    r = lambda *s: torch.randn(*s, generator=g, dtype=F64)
    f = lambda t: t.to(dtype).to(F64)
    C = 2 * G * dk + H * dv
    c = {"wconv": r(C, taps) * 0.7, "rate": torch.exp(r(H) * 1.5) if rate is None else torch.full((H,), rate, dtype=F64),
         "dt": r(H * dk if channel else H) * 1.5 - 1.0, "norm": r(dv) * 0.4 + 1.0, "eps": 1e-4}
    proj, z, want = {}, {}, {}
    for s, T in lens.items():
        proj[s] = f(torch.cat([r(T, C), r(T, H * dv), r(T, H) * 2, r(T, H) * 2], 1))     # q k v | gate | beta | decay
        z[s] = (r(T, H * dk) * 2).float().to(F64) if channel else None
        q, k, v = (pz.silu(pz.causal_conv(proj[s][:, :C], c["wconv"].float().to(F64)))[:, a:b]
                   for a, b in ((0, G * dk), (G * dk, 2 * G * dk), (2 * G * dk, C)))
        rep = lambda t: pz.unit_length(t.reshape(T, G, dk)).repeat_interleave(H // G, 1)
        logit = z[s] if channel else proj[s][:, C + H * dv + H:]
        lg = -c["rate"].repeat_interleave(dk if channel else 1) * pz.softplus(logit + c["dt"])
        decay = torch.exp(lg).view(T, H, -1).expand(T, H, dk)
        beta = torch.sigmoid(proj[s][:, C + H * dv:C + H * dv + H])
        o = pz.delta_rule(rep(q) * dk ** -0.5, rep(k), v.reshape(T, H, dv), decay, beta)
        gate = proj[s][:, C:C + H * dv]
        want[s] = (pz.unit_rms(o, c["eps"]) * c["norm"]).reshape(T, H * dv) * (torch.sigmoid(gate) if channel else pz.silu(gate))
    return c, proj, z, want


def _run_delta(ctx, rows, c, proj, z, state, H, G, dk, dv, channel, dtype):
    from glassbox_amd import ops
    C = 2 * G * dk + H * dv
    p = _dev(torch.cat([proj[s][a:b] for s, a, b in rows]), dtype)
    zz = _dev(torch.cat([z[s][a:b] for s, a, b in rows])) if channel else None
    n = p.shape[0]
    wide = torch.full((n, H * dv + 16), 9.0, dtype=dtype, device=DEV)
    gate = p[:, C:C + H * dv]
    ops.delta_rule(p, 0, C + H * dv, C + H * dv + H, _dev(c["wconv"].t()), _dev(c["rate"]), _dev(c["dt"]), zz, state, ctx, H, G, dk, dv,
                   gate, channel, _dev(c["norm"]), c["eps"], wide[:, 8:8 + H * dv])
    assert torch.all(wide[:, :8] == 9.0) and torch.all(wide[:, 8 + H * dv:] == 9.0)
    got, at = {}, 0
    for s, a, b in rows:
        got[(s, a)] = wide[at:at + b - a, 8:8 + H * dv].cpu().to(F64)
        at += b - a
    return got


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("H, G, dk, dv, taps, channel", DELTA_CASES)
def test_the_delta_rule_in_portions_of_a_batch(dtype, H, G, dk, dv, taps, channel):
    """Three requests whose tokens come in steps of single tokens, portions shorter than the convolution, portions at and
    around a chunk's 64 tokens and long ones, beside one another, into slots that hold garbage: every token against the
    plain recurrence over its whole sequence, in chunks (with ``tuned``) and token by token."""
    from glassbox_amd import ops
    lens = {0: 233, 1: 70, 2: 41}
    c, proj, z, want = _delta_inputs(lens, H, G, dk, dv, taps, channel, dtype, seed=H * dk + dv)
    cuts = [{0: 1, 1: 63, 2: 2}, {0: 64, 1: 1, 2: 1}, {0: 65, 2: 33}, {0: 2, 1: 2}, {0: 1, 1: 1, 2: 1}, {0: 100, 1: 3, 2: 4}]
    slots = {0: 2, 1: 0, 2: 3}
    floats, _ = ops.delta_slot(H, G, dk, dv, taps)
    for tuned in (True, False):
        state = torch.full((5, floats), 1e30, device=DEV)
        done = {s: 0 for s in lens}
        for cut in cuts:
            rows = sorted(((s, done[s], done[s] + m) for s, m in cut.items()), key=lambda r: (r[2] - r[1] != 1, r[0]))
            got = _run_delta(_step_ctx(rows, slots, tuned), rows, c, proj, z, state, H, G, dk, dv, channel, dtype)
            for s, a, b in rows:
                done[s] = b
                # (a head's output is divided by its own size: one that nearly cancels is as uncertain as its sum)
                tol = 2e-4 if dtype == torch.float32 else 4e-2
                err = (got[(s, a)] - want[s][a:b]).abs()
                assert err.max() < tol * float(want[s].abs().max()), (tuned, s, a, b)
        assert done == lens and torch.all(state[1] == 1e30) and torch.all(state[4] == 1e30)


@pytest.mark.parametrize("channel", [False, True])
def test_a_far_write_is_read_and_a_strong_decay_forgets_it(channel):
    """A value written at position 3 is read 900 tokens later, across chunks, portions and single tokens, when nothing decays; and
    with decays that take almost everything, chunks give what the token before alone leaves."""
    from glassbox_amd import ops
    H, G, dk, dv, taps = 2, 1, 64, 32, 2
    floats, _ = ops.delta_slot(H, G, dk, dv, taps)
    T = 910
    for rate in (0.0, 300.0):
        c, proj, z, want = _delta_inputs({0: T}, H, G, dk, dv, taps, channel, torch.float32, seed=5, rate=rate)
        C = 2 * G * dk + H * dv
        if rate == 0.0:   # no decay: after the first tokens nothing more is written (beta 0), and the queries look for position 3's key
            p = proj[0].clone()
            p[5:, C + H * dv:C + H * dv + H] = -200.0
            p[6:, :dk] = 0.0
            p[899:, :dk] = p[3, dk:2 * dk]
            p[898, :dk] = p[2, dk:2 * dk]
            c, proj, z, want = _again(c, {0: p}, z, H, G, dk, dv, channel)
            assert float(want[0][905:].abs().max()) > 0.1
        for cut in ([T], [300, 1, 2, 500, 97] + [1] * 10, [64] * 14 + [14]):
            state, at = torch.full((3, floats), 1e30, device=DEV), 0
            for m in cut:
                rows = [(0, at, at + m)]
                got = _run_delta(_step_ctx(rows, {0: 1}), rows, c, proj, z, state, H, G, dk, dv, channel, torch.float32)
                err = (got[(0, at)] - want[0][at:at + m]).abs().max()
                assert err < 2e-4 * float(want[0].abs().max()), (rate, at, m)
                at += m


def _again(c, proj, z, H, G, dk, dv, channel):
    """The plain results for projections that were changed."""
    want = {}
    C = 2 * G * dk + H * dv
    for s, p in proj.items():
        T = p.shape[0]
        q, k, v = (pz.silu(pz.causal_conv(p[:, :C], c["wconv"].float().to(F64)))[:, a:b]
                   for a, b in ((0, G * dk), (G * dk, 2 * G * dk), (2 * G * dk, C)))
        rep = lambda t: pz.unit_length(t.reshape(T, G, dk)).repeat_interleave(H // G, 1)
        logit = z[s] if channel else p[:, C + H * dv + H:]
        lg = -c["rate"].repeat_interleave(dk if channel else 1) * pz.softplus(logit + c["dt"])
        o = pz.delta_rule(rep(q) * dk ** -0.5, rep(k), v.reshape(T, H, dv), torch.exp(lg).view(T, H, -1).expand(T, H, dk),
                          torch.sigmoid(p[:, C + H * dv:C + H * dv + H]))
        gate = p[:, C:C + H * dv]
        want[s] = (pz.unit_rms(o, c["eps"]) * c["norm"]).reshape(T, H * dv) * (torch.sigmoid(gate) if channel else pz.silu(gate))
    return c, proj, z, want


# ------------------------------------------------------------------------------------------ whole models
_ORACLE = {}


def _requests(vocab, seed=0):
    return {r: helpers.random_tokens(vocab, n, seed=seed + n) for r, n in {"a": 130, "b": 47, "c": 1, "d": 71, "e": 2, "f": 24}.items()}


def _want(folder: str, tokens, dtype: str) -> np.ndarray:
    key = (folder, tuple(tokens), dtype)
    if key not in _ORACLE:
        cfg, w = pz.load_folder(folder)
        _ORACLE[key] = pz.forward(cfg, rounded(w) if dtype == "bfloat16" else w, list(tokens)).numpy()
    return _ORACLE[key]


SAMPLES = (1, 2, 3)


def _moved_by_rounding(folder: str, tokens) -> np.ndarray:
    """Root mean square over the vocabulary of what rounding the activations to bfloat16 moves each position's logits by: the
    largest of several ways of rounding."""
    key = (folder, tuple(tokens), "moved")
    if key not in _ORACLE:
        cfg, w = pz.load_folder(folder)
        want = _want(folder, tokens, "bfloat16")
        _ORACLE[key] = np.max([np.sqrt(((pz.forward(cfg, rounded(w), list(tokens), coarse=k).numpy() - want) ** 2).mean(1))
                               for k in SAMPLES], 0)
    return _ORACLE[key]


def _close_calls(folder: str, tokens) -> np.ndarray:
    """Positions at which some router's choice hangs on less than rounding to bfloat16 moves its logits by: a margin
    (``route_margin``) below ``ROUTE_TIMES`` times the most that rounding the activations, in several ways, moved that margin by
    in the plain implementation itself, or below ``ROUTE_MARGIN``.  There an engine that rounds may send the token to other
    experts than the plain implementation does, both being right; such positions are left out of the comparison in bfloat16."""
    key = (folder, tuple(tokens), "margins")
    if key not in _ORACLE:
        cfg, w = pz.load_folder(folder)
        fine, moved = [], None
        pz.forward(cfg, rounded(w), list(tokens), margins=fine)
        for k in SAMPLES:
            coarse = []
            pz.forward(cfg, rounded(w), list(tokens), margins=coarse, coarse=k)
            d = torch.stack([(a - b).abs().nan_to_num(0.0) for a, b in zip(fine, coarse)])
            moved = d if moved is None else torch.maximum(moved, d)
        _ORACLE[key] = (torch.stack(fine) < torch.clamp(ROUTE_TIMES * moved, min=ROUTE_MARGIN)).any(0).numpy()
    return _ORACLE[key]


ROUTE_MARGIN, ROUTE_TIMES = 3e-2, 2.5

#: A 32-bit engine is held to helpers.TOL_F32 of the request's largest logit at every position.  A bfloat16 engine is
#: compared with the plain implementation on the weights it holds by the root mean square of a position's logit
#: differences: at most 3 times what rounding the activations moves that position in the plain implementation itself, or
#: 1 % of the request's logits' root mean square where that is more.  One sample of rounding is no sharp bound on
#: another: a position's movement counts as at least the median over its request; no position may be beyond one and
#: a half times its limit, and one in fifty beyond the limit itself.
BF16_TIMES, BF16_FLOOR = 3.0, 1e-2


def _check(got, folder, requests, dtype, what):
    for r, toks in requests.items():
        want = _want(folder, toks, dtype)
        if dtype == "float32":
            tol = helpers.TOL_F32 * max(1.0, float(np.abs(want).max()))
            bad = helpers.first_bad(got[r], want, tol)
            assert bad is None, f"{what}, {dtype}, request {r} ({len(toks)} tokens): position {bad[0]} is {bad[1]:.3e} off (limit {tol:.3e})"
            continue
        err = np.sqrt(((got[r] - want) ** 2).mean(1))
        moved = _moved_by_rounding(folder, toks)
        lim = np.maximum(BF16_TIMES * np.maximum(moved, np.median(moved)), BF16_FLOOR * float(np.sqrt((want ** 2).mean())))
        close = _close_calls(folder, toks)
        assert close.sum() <= max(2, len(toks) // 4), f"{close.sum()} of {len(toks)} positions are close calls of a router"
        err = np.where(close, 0.0, err)
        # a token that went to other experts writes something else into the memories of the layers after: the positions
        # behind it that read that are moved too; they get six times the room
        lim = np.where(np.cumsum(close) > 0, 6.0 * lim, lim)
        over = np.nonzero(err > lim)[0]
        assert over.size <= max(1, len(toks) // 50) and float((err / lim).max()) <= 1.5, (
            f"{what}, {dtype}, request {r} ({len(toks)} tokens): position {over[0]} is {err[over[0]]:.3e} off "
            f"(limit {lim[over[0]]:.3e}); {over.size} positions over their limits, worst ratio {(err / lim).max():.2f}")


def _poison(engine) -> None:
    """Garbage in every page and state slot: whatever a request reads, it must have written itself."""
    for lc in engine.layers:
        for t in (lc.k_pages, lc.v_pages, lc.state):
            if t is not None:
                t.fill_(300)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", list(CASES))
def test_every_way_of_cutting_requests_into_steps(model_dirs, name, dtype):
    from glassbox_amd.engine import Engine
    folder = folder_of(model_dirs.base, name, calm=dtype == "bfloat16")
    requests = _requests(CASES[name]["vocab"])
    mixed, peak = helpers.schedule_mixed(requests, seed=3, live=3, tail=20)
    eng = Engine(folder, dtype=dtype, max_tokens=max(peak, 192), max_seqs=3)
    _poison(eng)
    for what, steps in (("whole", helpers.schedule_whole(requests)), ("last tokens one by one", helpers.schedule_tail(requests, 60)),
                        ("portions", helpers.schedule_chunks(requests)), ("portions of two", None), ("mixed batches", mixed)):
        if what == "portions of two":
            steps = helpers.schedule_chunks({r: t for r, t in requests.items() if len(t) < 80}, (2,))
        got = helpers.replay(eng, steps)
        _check(got, folder, {r: requests[r] for r in got}, dtype, what)
        assert eng.cache.num_seqs() == 0 and eng.cache.free_state_slots() == 3
        assert all(eng.cache.used_pages(g) == 0 for g in range(len(eng.group_keys)))
        eng.cache.check_invariants()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["A", "D"])
def test_long_prompts_whole_and_in_long_portions(model_dirs, name, dtype):
    """A prompt of 700 tokens: the runs of positions end many times, the state goes through many chunks, and the experts
    are run on their own tokens (many rows)."""
    from glassbox_amd.engine import Engine
    folder = folder_of(model_dirs.base, name, calm=dtype == "bfloat16")
    vocab = CASES[name]["vocab"]
    requests = {"long": helpers.random_tokens(vocab, 700, seed=23), "short": helpers.random_tokens(vocab, 40, seed=22)}
    eng = Engine(folder, dtype=dtype, max_tokens=1024, max_seqs=2)
    _poison(eng)
    for what, steps in (("whole", helpers.schedule_whole(requests)), ("long portions", helpers.schedule_chunks(requests, (300, 1, 399))),
                        ("a long portion beside single tokens", [
                            {"entries": [("short", requests["short"][:39], list(range(39)))], "end": []},
                            {"entries": [("long", requests["long"], list(range(700))), ("short", requests["short"][39:], [0])],
                             "end": ["long", "short"]}])):
        got = helpers.replay(eng, steps)
        _check(got, folder, requests, dtype, what)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_long_decoding(model_dirs, dtype):
    """250 tokens one by one after a prompt of four (runs and pages end many times over; in bfloat16 the steps are
    replayed from graphs)."""
    from glassbox_amd.engine import Engine
    folder = folder_of(model_dirs.base, "A", calm=dtype == "bfloat16")
    toks = helpers.random_tokens(211, 254, seed=11)
    steps = helpers.schedule_tail({"x": toks}, 250)
    eng = Engine(folder, dtype=dtype, max_tokens=320, max_seqs=2)
    _poison(eng)
    got = helpers.replay(eng, steps)
    if dtype == "bfloat16":
        assert eng.decode_graphs is not None and eng.decode_graphs.replays > 200
    _check(got, folder, {"x": toks}, dtype, "long decoding")
    plain = Engine(folder, dtype=dtype, max_tokens=320, max_seqs=2, graph_decode=False, kernels="plain")
    again = helpers.replay(plain, steps)
    _check(again, folder, {"x": toks}, dtype, "long decoding, plain kernels")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_layers_of_a_kind_are_made_again_from_the_launches_of_the_first(model_dirs, dtype):
    """Two kinds of layers, three times in turn: later ones of a kind are the first's launches with their own tensors, pages and
    state; the same bits as with every layer walked, and the plain implementation's logits."""
    from glassbox_amd import ops
    from glassbox_amd.engine import Engine
    folder = folder_of(model_dirs.base, "E", calm=dtype == "bfloat16")
    requests = {"a": helpers.random_tokens(97, 150, seed=1), "b": helpers.random_tokens(97, 41, seed=2)}
    steps = helpers.schedule_whole(requests) + helpers.schedule_chunks(requests, (70, 3, 40))
    before = ops.TAPE_COUNTS["replayed_layers"]
    taped = helpers.replay(Engine(folder, dtype=dtype, max_tokens=512, max_seqs=2), steps)
    assert ops.TAPE_COUNTS["replayed_layers"] >= before + len(steps)
    before = ops.TAPE_COUNTS["replayed_layers"]
    walked = helpers.replay(Engine(folder, dtype=dtype, max_tokens=512, max_seqs=2, layer_tapes=False), steps)
    assert ops.TAPE_COUNTS["replayed_layers"] == before
    assert all(np.array_equal(taped[r], walked[r]) for r in requests)
    whole = helpers.replay(Engine(folder, dtype=dtype, max_tokens=512, max_seqs=2), helpers.schedule_whole(requests))
    _check(whole, folder, requests, dtype, "layers made again")


def test_a_pool_that_holds_runs_not_requests(model_dirs):
    """A request of 600 tokens in a pool of 256: every attention of the model sees runs of 40 positions, and the pages of a run
    that has ended go back to the pool while the request lives (portions of 100, then single tokens)."""
    from glassbox_amd.engine import Engine
    folder = folder_of(model_dirs.base, "E")
    toks = helpers.random_tokens(97, 600, seed=31)
    eng = Engine(folder, dtype="float32", max_tokens=256, max_seqs=2)
    _poison(eng)
    steps = helpers.schedule_chunks({"x": toks[:520]}, (100,))
    steps[-1]["end"] = []
    steps += [{"entries": [("x", [t], [0])], "end": ["x"] if i == 79 else []} for i, t in enumerate(toks[520:])]
    got = helpers.replay(eng, steps)
    _check(got, folder, {"x": toks}, "float32", "a pool smaller than its request")
    assert all(eng.cache.used_pages(g) == 0 for g in range(len(eng.group_keys)))


def test_slots_and_pages_that_are_used_again(model_dirs):
    """Two slots, six requests one after the other in pairs: a request finds the slot (the memory and the convolution's last rows) and the
    pages of one that ended, and must start from nothing."""
    from glassbox_amd.engine import Engine
    folder = folder_of(model_dirs.base, "D")
    requests = {r: helpers.random_tokens(160, n, seed=70 + n) for r, n in {"p": 50, "q": 31, "r": 18, "s": 64, "t": 2, "u": 45}.items()}
    eng = Engine(folder, dtype="float32", max_tokens=128, max_seqs=2)
    _poison(eng)
    steps, _ = helpers.schedule_mixed(requests, seed=5, live=2, tail=6)
    got = helpers.replay(eng, steps)
    _check(got, folder, requests, "float32", "slots used again")


def test_batches_of_unequal_requests_give_each_what_it_gets_alone(model_dirs):
    """In 32-bit a request's logits do not depend on what else is in its batch, beyond rounding of the sums' order."""
    from glassbox_amd.engine import Engine
    folder = folder_of(model_dirs.base, "B")
    requests = _requests(130, seed=4)
    eng = Engine(folder, dtype="float32", max_tokens=1024, max_seqs=6)
    alone = helpers.replay(eng, helpers.schedule_whole(requests))
    together = helpers.replay(eng, [{"entries": [(r, t, list(range(len(t)))) for r, t in requests.items()], "end": list(requests)}])
    for r in requests:
        assert np.abs(alone[r] - together[r]).max() < 2e-5 * max(1.0, float(np.abs(alone[r]).max()))


# ------------------------------------------------------------------------------------------ generation
def _greedy(cfg, w, prompt, n):
    toks = list(prompt)
    for _ in range(n):
        toks.append(int(torch.argmax(pz.forward(cfg, w, toks)[-1])))
    return toks[len(prompt):]


@pytest.mark.parametrize("name", ["A", "E"])
def test_greedy_generation_through_the_entry_points(model_dirs, name):
    from glassbox_amd.engine import Engine, generate, greedy
    folder = folder_of(model_dirs.base, name, seed=2)
    cfg, w = pz.load_folder(folder)
    vocab = CASES[name]["vocab"]
    prompts = [helpers.random_tokens(vocab, n, seed=50 + n) for n in (5, 44, 1, 23, 70)]
    want = [_greedy(cfg, w, p, 12) for p in prompts]
    assert len({tuple(r) for r in want}) > 2, "replies that do not depend on the prompt show nothing"
    eng = Engine(folder, dtype="float32", max_tokens=1024, max_seqs=3)
    assert greedy(eng, prompts[1], 12) == want[1]
    # the scheduler: three live requests at most, prompts in portions of at most 16 tokens beside decoding requests
    assert generate(eng, prompts, max_tokens=12, token_budget=16, max_seqs=3) == want
    assert eng.cache.num_seqs() == 0 and eng.cache.free_state_slots() == 3


def test_the_command_line_runs_the_model(model_dirs, tmp_path):
    folder = folder_of(model_dirs.base, "B", seed=2)
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    run = lambda *args, stdin=None: subprocess.run([sys.executable, os.path.join(root, "bin", "glassbox"), *args],
                                                   capture_output=True, text=True, timeout=600, input=stdin)
    r = run("generate", "--model", folder, "--prompt", "5,17,3,99,41", "-n", "8", "--dtype", "float32", "--no-prefix-cache")
    assert r.returncode == 0, r.stderr
    cfg, w = pz.load_folder(folder)
    assert [int(t) for t in r.stdout.split()] == _greedy(cfg, w, [5, 17, 3, 99, 41], 8)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": [5, 17, 3, 9], "want": [1, 3]}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": [8], "want": [0]}, {"id": "b", "tokens": [4, 4], "want": []}], "end": ["a"]}]
    r = subprocess.run([os.path.join(root, "bin", "trace_run"), "--model", folder, "--dtype", "float32", "--out", str(tmp_path / "o"),
                        "--max-tokens", "128"], capture_output=True, text=True, timeout=600,
                       input="".join(json.dumps(s) + "\n" for s in steps))
    assert r.returncode == 0 and r.stdout.split() == ["done", "0", "done", "1"], r.stderr
    want = pz.forward(cfg, w, [5, 17, 3, 9, 8]).numpy()
    assert np.abs(np.fromfile(tmp_path / "o" / "0.f32", dtype="<f4").reshape(2, -1) - want[[1, 3]]).max() < 1e-4
    assert np.abs(np.fromfile(tmp_path / "o" / "1.f32", dtype="<f4") - want[4]).max() < 1e-4
