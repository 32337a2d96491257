"""Zakusun on the device: each mechanism's kernels against the plain implementation, then whole models under every
way of cutting requests into steps, and generation through the entry points."""
from __future__ import annotations

import json
import math
import os
import subprocess
import sys
from types import SimpleNamespace

import numpy as np
import pytest
import torch

import helpers
from plain import zakusun as pz
from zakusun_cases import CASES, folder_of, rounded

pytestmark = pytest.mark.gpu
F64 = torch.float64
DEV = "cuda:0"
DTYPES = [torch.float32, torch.bfloat16]


def _dev(t, dtype=torch.float32):
    return t.to(dtype).to(DEV).contiguous()


def _i32(values):
    return torch.tensor(list(values), dtype=torch.int32, device=DEV)


def _step_ctx(rows, slots=None, dtype=torch.float32, tuned=True, page_size=16, tables=None, cache_rows=None):
    """The tables of a step whose requests bring ``rows`` = [(request, first position, end position)], in that order (single
    tokens first).  ``tables``, ``cache_rows``: by request, its block table and the cache row of each position."""
    from glassbox_amd.engine.context import Workspace
    lens = [b - a for _, a, b in rows]
    starts = np.cumsum([0] + lens)[:-1]
    tok_seq = [s for s, n in enumerate(lens) for _ in range(n)]
    ctx = SimpleNamespace(n=sum(lens), dtype=dtype, tuned=tuned, fuse_norms=tuned, page_size=page_size, memo={}, num_seqs=len(rows),
                          positions=_i32(p for _, a, b in rows for p in range(a, b)), tok_seq=_i32(tok_seq),
                          q_start=_i32(starts), q_len=_i32(lens), pos0=_i32(a for _, a, _ in rows),
                          state_slots=_i32((slots[r] if slots else 0) for r, _, _ in rows),
                          host={"max_q_len": max(lens), "n_decode": sum(1 for n in lens if n == 1), "q_len": lens,
                                "pos0": [a for _, a, _ in rows], "max_context": max(b for _, _, b in rows)},
                          buffer=Workspace(torch.device(DEV)).buffer)
    if tables is not None:
        width = max(len(tables[r]) for r, _, _ in rows)
        ctx.tables = [_i32(v for r, _, _ in rows for v in tables[r] + [-1] * (width - len(tables[r]))).view(len(rows), width)]
        ctx.slots = [_i32(cache_rows[r][p] for r, a, b in rows for p in range(a, b))]
    return ctx


def _pages(lens, P, seed=0, spare=3):
    """Block tables and cache rows for requests of ``lens`` tokens that share one shuffled pool; (tables, rows, pages)."""
    need = {r: -(-T // P) for r, T in lens.items()}
    total = sum(need.values()) + spare
    order = np.random.RandomState(seed).permutation(total).tolist()
    tables, rows, at = {}, {}, 0
    for r, T in lens.items():
        tables[r] = order[at:at + need[r]]
        at += need[r]
        rows[r] = [tables[r][p // P] * P + p % P for p in range(T)]
    return tables, rows, total


# ------------------------------------------------------------------------------------------ embedding
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("d, copies", [(64, 2), (50, 1), (7, 2), (1030, 3)])
def test_embedded_rows_with_the_vector_of_their_position(d, copies, dtype):
    from glassbox_amd.parts.embedding import SinusoidEmbedding
    torch.manual_seed(d)
    vocab = 40
    table = torch.randn(vocab, d)
    part = SinusoidEmbedding(vocab, d)
    part.load({"weight": _dev(table, dtype)})
    positions = [0, 1, 2, 63, 64, 1000, 8191, 131071, 1000003]
    ids = [(7 * i) % vocab for i in range(len(positions))]
    out = torch.empty(copies, len(ids), d, device=DEV)
    part.forward(SimpleNamespace(token_ids=_i32(ids), positions=_i32(positions)), out)
    want = table.to(dtype).to(F64)[ids] + pz.sinusoid(torch.tensor(positions), d)
    for k in range(copies):
        assert (out[k].cpu().to(F64) - want).abs().max() < 1e-6


# ------------------------------------------------------------------------------------------ norms, convolutions, sums over depth
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("n, d, groups", [(5, 64, 2), (3, 50, 5), (700, 96, 3), (2, 2048, 4), (3, 5000, 1), (9, 24, 3), (600, 1500, 5),
                                          (4, 8192, 8), (2, 9000, 9), (1, 320, 64)])
def test_one_pass_adds_a_sublayer_sums_over_depth_and_norms_in_groups(n, d, groups, dtype):
    """Every combination of what the pass may do, against the plain functions; groups of very different sizes."""
    from glassbox_amd import ops
    torch.manual_seed(n + d)
    eps, tol = 1e-5, (3e-6 if dtype == torch.float32 else 1e-2)
    x = (torch.randn(n, groups, d // groups) * torch.logspace(-2, 2, groups)[None, :, None]).reshape(n, d).float()
    gamma = torch.randn(d).float()
    y = torch.randn(3, n, d).float()
    for slices in (0, 1, 3):
        for count in (0, 1, 6):
            hist = torch.randn(max(count, 1), n, d).float()
            coef = torch.randn(count + 1).float()
            res = _dev(x)
            out = torch.full((n, d), 9.0, device=DEV)
            h = torch.empty(n, d, dtype=dtype, device=DEV)
            scales = torch.empty(n, groups, device=DEV)
            ops.residual_rows(res, _dev(y[:slices]) if slices > 1 else _dev(y[0]) if slices else None, max(slices, 1),
                              (_dev(hist), _dev(coef), out) if count else None, _dev(gamma), groups, eps, scales=scales, h=h)
            new = x.to(F64) + (y[:slices].to(F64).sum(0) if slices else 0.0)
            assert (res.cpu().to(F64) - new).abs().max() < 2e-6 * float(new.abs().max()), (slices, count)
            went = new
            if count:
                went = pz.depth_average(coef.to(F64), [hh.to(F64) for hh in hist] + [new])
                assert (out.cpu().to(F64) - went).abs().max() < 3e-6 * float(went.abs().max() + hist.abs().max() * coef.abs().max()), (slices, count)
            else:
                assert torch.all(out == 9.0)
            seen = out if count else res     # (the norm of what the pass left, in its own 32 bits)
            want = pz.group_norm(seen.cpu().to(F64), gamma.to(F64), groups, eps)
            assert (h.cpu().to(F64) - want).abs().max() < tol * float(want.abs().max()), (slices, count)
            apart = torch.empty(n, d, dtype=dtype, device=DEV)
            ops.norm_conv(seen, scales, _dev(gamma), None, None, _step_ctx([(0, 0, n)]), apart)
            assert (apart.float() - h.float()).abs().max() <= (1e-6 if dtype == torch.float32 else 1e-2) * float(want.abs().max())
    picked = [n - 1, 0, n // 2]
    rows = torch.empty(3, d, dtype=dtype, device=DEV)
    ops.residual_rows(_dev(x), gamma=_dev(gamma), groups=groups, eps=eps, h=rows, rows=_i32(picked))
    want = pz.group_norm(x.to(F64), gamma.to(F64), groups, eps)[picked]
    assert (rows.cpu().to(F64) - want).abs().max() < tol * float(want.abs().max())


@pytest.mark.parametrize("tuned", [True, False])
@pytest.mark.parametrize("d, groups, taps, dtype", [(64, 2, 4, torch.float32), (50, 5, 2, torch.bfloat16), (24, 3, 8, torch.float32),
                                                    (16, 1, 1, torch.float32), (40, 2, 0, torch.bfloat16), (96, 4, 5, torch.bfloat16),
                                                    (7, 7, 3, torch.float32), (2048, 8, 4, torch.bfloat16)])
def test_normed_rows_and_their_convolution_in_portions_of_a_batch(d, groups, taps, dtype, tuned):
    """Three requests whose tokens come in four steps of unequal portions (single tokens, portions shorter than the
    convolution, long ones; the first and third steps bring single tokens only, so one pass does it all) into slots that
    hold garbage, the second of two convolutions that share a slot: rows against the plain functions on whole sequences,
    the slots after every step, and the other convolution's rows untouched."""
    from glassbox_amd.parts.base import LayerCache
    from glassbox_amd.parts.conv import ConvolvedNorm
    from glassbox_amd.parts.norm import GroupRMSNorm
    torch.manual_seed(d + taps)
    eps = 1e-5
    lens = {0: 23, 1: 3, 2: 9}
    cuts = {0: (1, 20, 1, 1), 1: (1, 1, 0, 1), 2: (1, 2, 1, 5)}
    slots = {0: 2, 1: 0, 2: 3}
    part = ConvolvedNorm(GroupRMSNorm(d, groups, eps), taps, place=1)
    gamma, w = torch.randn(d).float(), torch.randn(d, taps).float() if taps else None
    part.norm.load({"weight": _dev(gamma)})
    part.load({"conv": _dev(w)} if taps else {})
    state = torch.full((5, 2, max(taps - 1, 1), d), 55.0, device=DEV) if taps > 1 else None
    x = {r: torch.randn(T, d).float() for r, T in lens.items()}
    add = {r: torch.randn(2, T, d).float() for r, T in lens.items()}
    res = {r: x[r].to(F64) + add[r].to(F64).sum(0) for r in lens}
    normed = {r: pz.group_norm(res[r], gamma.to(F64), groups, eps) for r in lens}
    want = {r: pz.with_conv(normed[r], w.to(F64) if taps else None) for r in lens}
    tol = 1e-5 if dtype == torch.float32 else 1e-2
    done = {r: 0 for r in lens}
    for step in range(4):
        rows = [(r, done[r], done[r] + cuts[r][step]) for r in lens if cuts[r][step]]
        rows.sort(key=lambda v: v[2] - v[1] > 1)
        ctx = _step_ctx(rows, slots, dtype, tuned)
        xs = _dev(torch.cat([x[r][a:b] for r, a, b in rows], 0))
        ys = _dev(torch.cat([add[r][:, a:b] for r, a, b in rows], 1))
        got = part.after(ctx, xs, LayerCache(state=state), ys, 2).cpu().to(F64)
        at = 0
        for r, a, b in rows:
            assert (got[at:at + b - a] - want[r][a:b]).abs().max() < tol * float(want[r].abs().max()), (step, r)
            at += b - a
            done[r] = b
            if state is not None:
                kept = state[slots[r], 1].cpu().to(F64)
                for i in range(taps - 1):
                    p = b - (taps - 1) + i
                    if p >= 0:
                        assert (kept[i] - normed[r][p]).abs().max() < 1e-5 * float(normed[r].abs().max()), (step, r, i)
    if state is not None:
        assert torch.all(state[:, 0] == 55.0) and torch.all(state[1] == 55.0) and torch.all(state[4] == 55.0)


# ------------------------------------------------------------------------------------------ latents and their pages
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("R, P", [(96, 16), (40, 32), (512, 16), (18, 16), (7, 48), (520, 16)])
def test_latents_into_pages_and_back_as_rows(R, P, dtype):
    """Normed latents land in their cache rows and nowhere else; the gathered rows of two portions' contexts are what was
    stored, with zeros behind a context's end although the page holds other things there."""
    from glassbox_amd import ops
    torch.manual_seed(R)
    lens = {0: 37, 1: 70}
    tables, rows, pages = _pages(lens, P, seed=R)
    c_pages = torch.full(ops.key_pages_shape(pages, 1, P, R), float("nan"), dtype=dtype, device=DEV)
    gamma = torch.randn(R).float()
    raw = {r: (torch.randn(T, R + 5) * 3).to(dtype) for r, T in lens.items()}
    want = {r: pz.unit_rms(raw[r][:, :R].to(F64), 1e-5) * gamma.to(F64) for r in lens}
    wide = torch.cat([raw[0], raw[1]], 0)
    if (R + 5) % 8:
        wide = torch.cat([wide, torch.zeros(wide.shape[0], 8 - (R + 5) % 8, dtype=dtype)], 1)
    ops.latent_store(wide.to(DEV)[:, :R], _dev(gamma), 1e-5, _i32(rows[0] + rows[1]), c_pages)
    stored = ops.unpack_keys(c_pages).reshape(pages * P, R).cpu().to(F64)
    tol = 2e-6 if dtype == torch.float32 else 1e-2
    for r in lens:
        assert (stored[rows[r]] - want[r]).abs().max() < tol * float(want[r].abs().max())
    others = sorted(set(range(pages * P)) - set(rows[0]) - set(rows[1]))
    assert torch.isnan(stored[others]).all()
    ctx = _step_ctx([("d", 3, 4), (0, 20, 37), (1, 0, 70)], tables=dict(tables, d=[0]), cache_rows=dict(rows, d=[0] * 8))
    need = [-(-37 // P), -(-70 // P)]
    table = torch.full((3, max(need)), -7, dtype=torch.int32, device=DEV)
    source = torch.full((sum(need), 2), -7, dtype=torch.int32, device=DEV)
    ops.latent_tables(ctx, 1, P, table, source)
    assert table[1, :need[0]].tolist() == list(range(need[0])) and table[2, :need[1]].tolist() == list(range(need[0], sum(need)))
    assert source.tolist() == [[1, i] for i in range(need[0])] + [[2, i] for i in range(need[1])]
    out = torch.full((sum(need) * P, R), 3.0, dtype=dtype, device=DEV)
    ops.latent_gather(c_pages, ctx.tables[0], source, ctx, out)
    got, at = out.cpu().to(F64), 0
    for r in lens:
        T = lens[r]
        assert torch.equal(got[at:at + T], stored[rows[r]])
        assert float(got[at + T:at + need[r] * P].abs().sum()) == 0.0
        at += need[r] * P


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H, hc, P", [(3, 64, 16), (5, 48, 32), (2, 136, 16), (1, 8, 64), (2, 264, 16)])
def test_rows_of_key_and_value_heads_into_scratch_pages(H, hc, P, dtype):
    from glassbox_amd import ops
    torch.manual_seed(hc)
    total = 3
    kv = torch.randn(total * P, 2 * H * hc).to(dtype)
    k_pages = torch.empty(ops.key_pages_shape(total, H, P, hc), dtype=dtype, device=DEV)
    v_pages = torch.empty((total, H, hc, P), dtype=dtype, device=DEV)
    ops.latent_expand(kv.to(DEV), k_pages, v_pages)
    keys = kv[:, :H * hc].view(total, P, H, hc).permute(0, 2, 1, 3)
    values = kv[:, H * hc:].view(total, P, H, hc).permute(0, 2, 3, 1)
    assert torch.equal(ops.unpack_keys(k_pages).cpu(), keys) and torch.equal(v_pages.cpu(), values)


# ------------------------------------------------------------------------------------------ attention to the latents
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H, dk, dv, R, P", [(6, 24, 32, 96, 16), (16, 16, 16, 128, 32), (17, 8, 8, 136, 16), (3, 48, 64, 256, 16),
                                             (33, 8, 24, 264, 16), (32, 64, 64, 512, 16), (5, 40, 16, 512, 64), (2, 10, 6, 18, 16),
                                             (4, 16, 16, 520, 16), (1, 136, 72, 24, 16)])
def test_single_tokens_attend_to_latents(H, dk, dv, R, P, dtype):
    """Requests of 1 to 1,400 tokens decoded at the ends and edges of pages and of the chunks that workgroups take.  One
    latent a request is made to carry the softmax of a head: the first, the last, the ones at a page's and a chunk's edge,
    one far back; sinks take a visible share; unused rows of the pages are no numbers.  The tuned and the plain kernel
    against the plain functions on expanded keys and values."""
    from glassbox_amd import ops
    from glassbox_amd.engine.context import Workspace
    from glassbox_amd.parts.attention import cache_head_cols
    g = torch.Generator().manual_seed(H * R + dk)
    f = lambda t: t.to(dtype).to(F64)
    hc, scale = cache_head_cols(dk, dv), 0.5
    lens = {0: 1, 1: P, 2: P + 1, 3: 64, 4: 129, 5: 257, 6: 700, 7: 1400}
    tables, rows, pages = _pages(lens, P, seed=R + H)
    c_pages = torch.full(ops.key_pages_shape(pages, 1, P, R), float("nan"), dtype=dtype)
    flat = ops.unpack_keys(c_pages).reshape(pages * P, R).clone()
    uk, uv = f(torch.randn(H, dk, R, generator=g, dtype=F64) / R ** 0.5), f(torch.randn(H, dv, R, generator=g, dtype=F64) / R ** 0.5)
    c = {r: f(torch.randn(T, R, generator=g, dtype=F64)) for r, T in lens.items()}
    q = torch.randn(len(lens), H, dk, generator=g, dtype=F64) * 0.3
    sinks = torch.linspace(-2.0, 3.0, H, dtype=F64)
    for r, T in lens.items():
        flat[rows[r]] = c[r].to(dtype)
        for h in range(H):
            target = [0, T - 1, max(T - 1 - T % P, 0), T // 2, min(127, T - 1), min(128, T - 1), max(T - 600, 0), P - 1 if P <= T else 0][(h + r) % 8]
            key = uk[h] @ c[r][target]
            q[r, h] += 11.0 * key / (scale * float(key @ key))
    q = f(q)
    want = torch.zeros(len(lens), H, dv, dtype=F64)
    for r, T in lens.items():
        k, v = torch.einsum("hdr,tr->thd", uk, c[r]), torch.einsum("hdr,tr->thd", uv, c[r])
        s = torch.einsum("hd,thd->ht", q[r], k) * scale
        top = torch.maximum(s.max(-1).values, sinks)
        e = torch.exp(s - top[:, None])
        p = e / (e.sum(-1) + torch.exp(sinks - top))[:, None]
        if T > 1:
            assert float(p.max(-1).values.max()) > 0.35    # some head found its key
        want[r] = torch.einsum("ht,thd->hd", p, v)
    c_pages = ops.pack_keys(flat.view(pages, 1, P, R)).to(DEV)
    gate = torch.randn(len(lens), H * dv, generator=g, dtype=F64)
    want = want.reshape(len(lens), -1) * torch.sigmoid(f(gate))
    pad = lambda t, d: torch.cat([t, torch.zeros(*t.shape[:1], hc - d, *t.shape[2:], dtype=F64)], 1)
    uk_d = _dev(pad(uk, dk).reshape(H * hc, R), dtype)
    uv_d = _dev(pad(uv, dv).reshape(H * hc, R), dtype)
    uk_t = uk_d.view(H, hc, R).transpose(1, 2).contiguous()
    q_d = torch.zeros(len(lens), H, hc, dtype=dtype, device=DEV)
    q_d[:, :, :dk] = _dev(q, dtype)
    q_d = q_d.view(len(lens), H * hc)
    ctx = _step_ctx([(r, T - 1, T) for r, T in lens.items()], tables=tables, cache_rows=rows)
    ws = Workspace(torch.device(DEV))
    tol = 3e-5 if dtype == torch.float32 else 2.5e-2
    forms = [("plain", True)] + ([("tuned", False)] if ops.latent_tuned_takes(dtype, R, P) else [])
    if dtype == torch.bfloat16 and R % 8 == 0 and R <= 512:
        assert len(forms) == 2
    for name, plain in forms:
        ql = torch.empty(len(lens), H * R, dtype=dtype, device=DEV)
        ops.latent_absorb(q_d, uk_d, None if plain else uk_t, hc, dk, ql, H)
        absorbed = torch.einsum("nhd,hdr->nhr", q, uk).reshape(len(lens), -1)
        assert (ql.cpu().to(F64) - absorbed).abs().max() < tol * float(absorbed.abs().max()), name
        for max_context in (1400, 4096):      # (a replayed step's tables are made for longer contexts than it has)
            out = torch.full((len(lens), H * dv), 9.0, dtype=dtype, device=DEV)
            ops.latent_decode(ql, c_pages, ctx.tables[0], ctx.positions, ctx.tok_seq, H, scale, max_context, _dev(sinks), uv_d, hc, dv,
                              _dev(gate, dtype), out, ws.buffer, plain=plain)
            err = (out.cpu().to(F64) - want).abs().max(1).values
            assert float(err.max()) < tol * max(1.0, float(want.abs().max())), (name, max_context, err.tolist())


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H, dk, dv, R", [(3, 16, 24, 40), (2, 32, 32, 128), (2, 40, 48, 264), (2, 6, 10, 18), (1, 264, 24, 64)])
def test_the_mixer_finds_far_keys_in_prompts_in_portions_and_decoded(H, dk, dv, R, dtype):
    """The mixer alone on one request of 400 tokens whose hidden rows are made so that queries find single keys: the first
    token, the token before, the last of the page before, one far back (and a key just after the query, which must not be
    seen); a second request beside it.  Whole, in portions cut anywhere down to two tokens, and token by token."""
    from glassbox_amd.parts.attention import LatentCacheAttention
    from glassbox_amd.parts.base import LayerCache
    from glassbox_amd import ops
    torch.manual_seed(R)
    width, eps, P, scale, T = 280, 1e-5, 16, 0.4, 400
    part = LatentCacheAttention(width, H, dk, dv, R, scale, eps, sink=True)
    f = lambda t: t.to(dtype).to(F64)
    w = {n: (torch.randn(s.shape, dtype=F64) / max(1, s.shape[-1]) ** 0.5 if len(s.shape) == 2 else torch.randn(s.shape, dtype=F64).float().to(F64))
         for n, s in part.tensor_specs().items()}
    w = {n: f(t) if t.dim() == 2 else t for n, t in w.items()}
    part.load({n: _dev(t, dtype if t.dim() == 2 else torch.float32) for n, t in w.items()})
    named = {"x." + n: t for n, t in w.items()}
    hidden = {0: f(torch.randn(T, width, dtype=F64)), 1: f(torch.randn(90, width, dtype=F64))}
    back = torch.linalg.pinv(w["q"])                      # the hidden row whose queries are given
    c = pz.latent(named, "x.", eps, hidden[0])
    k = (c @ w["uk"].T).view(T, H, dk)
    plans = {}
    for i in range(33, T, 9):
        target = [0, i - 1, i - 1 - i % P, i - 31, min(i + 1, T - 1)][(i // 9) % 5]
        if target % 9 == 33 % 9 and target >= 33:
            continue                                       # (its own hidden row is changed too)
        pull = 8.0 * k[target] / (scale * (k[target] ** 2).sum(-1, keepdim=True))
        plans[i] = (target, back @ pull.reshape(-1))
    for i, (_, row) in plans.items():
        hidden[0][i] = f(row)
    m = {"heads": H, "dim": dk, "vdim": dv, "kv_rank": R, "scale": scale}
    want = {r: pz.latent_attention(named, "x.", m, eps, h) for r, h in hidden.items()}
    coarse = {r: pz.latent_attention(named, "x.", m, eps, h, pz.bf16) for r, h in hidden.items()}
    tables, cache_rows, pages = _pages({0: T, 1: 90}, P, seed=3)
    limit = {r: 3e-5 * float(want[r].abs().max()) if dtype == torch.float32 else
             4.0 * float((coarse[r] - want[r]).abs().max()) for r in want}
    for tuned in (True, False):
        cuts = {"whole": [T], "portions": [7, 2, 40, 16, 17, 100, 2, 31, 185], "tail": [300] + [1] * 100}
        for what, sizes in cuts.items():
            cache = LayerCache(torch.full(ops.key_pages_shape(pages, 1, P, R), float("nan"), dtype=dtype, device=DEV))
            at, other = 0, 0
            for s, size in enumerate(sizes):
                step = [(0, at, at + size)]
                if s % 3 != 1 and other < 90:              # the second request comes along in two steps of three
                    take = min(90 - other, 1 if s % 2 else 29)
                    step.append((1, other, other + take))
                    other += take
                step.sort(key=lambda v: v[2] - v[1] > 1)
                ctx = _step_ctx(step, None, dtype, tuned, P, tables, cache_rows)
                h = _dev(torch.cat([hidden[r][a:b] for r, a, b in step], 0), dtype)
                y = torch.full((h.shape[0], width), 5.0, device=DEV)
                made, slices = part.forward(ctx, h, y, cache, store=True)
                got = (made if slices == 1 else made[:slices * y.numel()].view(slices, *y.shape).sum(0)).cpu().to(F64)
                row = 0
                for r, a, b in step:
                    err = (got[row:row + b - a] - want[r][a:b]).abs().max(1).values
                    assert float(err.max()) < limit[r], (what, tuned, r, a, b, int(err.argmax()) + a, float(err.max()), limit[r])
                    row += b - a
                at += size


# ------------------------------------------------------------------------------------------ the router and the experts
@pytest.mark.parametrize("E, top", [(6, 2), (8, 4), (16, 3), (4, 4), (3, 1), (64, 6), (65, 5), (130, 16), (300, 8)])
def test_the_router_chooses_by_logits_with_bias(E, top):
    from glassbox_amd import ops
    torch.manual_seed(E + top)
    n = 301
    z, bias = torch.randn(n, E + 2) * 2, torch.randn(E)
    z[7, :E] = -80.0          # far apart: the weights of the others vanish
    z[7, 1] = 80.0
    logits = z[:, :E].to(F64) + bias.to(F64)
    ids_w, wts_w = pz.route(logits, top)
    combine = torch.empty(n, E, device=DEV)
    ids, wts = torch.empty(n, top, dtype=torch.int32, device=DEV), torch.empty(n, top, device=DEV)
    ops.moe_route(_dev(z)[:, :E], E, _dev(bias), top, 1.0, False, combine, ids, wts, softmax="chosen")
    same = 0
    for t in range(n):
        if ids[t].tolist() != ids_w[t].tolist():   # only where two logits are as good as equal in 32-bit
            assert float(pz.route_margin(logits[t:t + 1], top)) < 1e-5 or set(ids[t].tolist()) == set(ids_w[t].tolist()), t
            continue
        same += 1
        assert (wts[t].cpu().to(F64) - wts_w[t]).abs().max() < 2e-6
        row = torch.zeros(E, dtype=F64)
        row[ids_w[t]] = wts_w[t]
        assert (combine[t].cpu().to(F64) - row).abs().max() < 2e-6
    assert same > n - 5


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("E, top, d", [(6, 2, 64), (64, 16, 40), (3, 3, 50), (12, 4, 2048), (1, 1, 8)])
def test_logits_and_route_in_one_kernel(E, top, d, dtype):
    """The same choice and weights as the product and the route kernel give, for rows of one to hundreds of tokens."""
    from glassbox_amd import ops
    torch.manual_seed(E + d)
    for n in (1, 9, 300):
        h, w, bias = torch.randn(n, d).to(dtype), (torch.randn(E, d) * 3 / d ** 0.5).to(dtype), torch.randn(E)
        z = h.to(F64) @ w.to(F64).T + bias.to(F64)
        ids_w, wts_w = pz.route(z, top)
        combine = torch.full((n, E), 9.0, device=DEV)
        ids, wts = torch.empty(n, top, dtype=torch.int32, device=DEV), torch.empty(n, top, device=DEV)
        ops.moe_router(h.to(DEV), w.to(DEV), _dev(bias), top, 0.5, combine, ids, wts)
        clear = pz.route_margin(z, top) > 1e-4
        assert clear.sum() > 0.9 * n
        dense = torch.zeros(n, E, dtype=F64).scatter_(1, ids_w, 0.5 * wts_w)
        assert (combine.cpu().to(F64) - dense)[clear].abs().max() < 5e-5
        given = torch.zeros(n, E, dtype=F64).scatter_(1, ids.cpu().long(), wts.cpu().to(F64))
        assert torch.equal(given, combine.cpu().to(F64))
        ordered = wts.cpu()
        assert torch.all(ordered[:, :-1] >= ordered[:, 1:])      # the largest logit's expert first


def test_grouped_products_by_tiles_of_256_rows_with_k_divided():
    """Rows of groups of very unequal size (none, one, a tile and a row more, several tiles) through the ring kernel: stored,
    behind the clamped unit, and with k divided into slices that are added, against the product by tiles of 128 rows."""
    from glassbox_amd import ops
    torch.manual_seed(6)
    d, ff, E = 256, 320, 5
    sizes = [0, 1, 257, 900, 300]
    n = sum(sizes)
    ids = torch.cat([torch.full((s,), e) for e, s in enumerate(sizes)])[torch.randperm(n)].int().view(n, 1)
    h = torch.randn(n, d).bfloat16().to(DEV)
    up = (torch.randn(2 * E * ff, d) * 0.1).bfloat16().to(DEV)
    down = (torch.randn(d, E * ff) * 0.1).bfloat16().to(DEV)
    got = {}
    for rows in (128, 256):
        tiles = ops.moe_sort_tiles(n, E, rows)
        counts, order = torch.empty(E, dtype=torch.int32, device=DEV), torch.empty(n, dtype=torch.int32, device=DEV)
        pos, tile_map = torch.empty(n, 1, dtype=torch.int32, device=DEV), torch.empty(tiles, 3, dtype=torch.int32, device=DEV)
        ops.moe_sort(ids.to(DEV), E, rows, counts, order, pos, tile_map)
        act = torch.full((n, ff), 7.0, dtype=torch.bfloat16, device=DEV)
        ops.gemm_grouped(h, order, up, ff * d, 2 * ff, tile_map, rows, act, silu_mul=True, up_offset=E * ff, unit=(1.0, 1.702, 1.0))
        plain = torch.full((n, ff), 7.0, dtype=torch.bfloat16, device=DEV)
        ops.gemm_grouped(h, order, up, ff * d, ff, tile_map, rows, plain)
        y = torch.full((n, d), 7.0, device=DEV)
        ops.gemm_grouped(act, None, down, ff, d, tile_map, rows, y)
        got[rows] = (act.float(), plain.float(), y)
        if rows == 256:
            for slices in (2, 3):
                parts = torch.full((slices, n, d), 7.0, device=DEV)
                ops.gemm_grouped(act, None, down, ff, d, tile_map, rows, parts)
                assert (parts.sum(0) - y).abs().max() < 1e-4 * float(y.abs().max())
                one, two = torch.zeros(n, d, device=DEV), torch.zeros(n, d, device=DEV)
                wts = torch.rand(n, 1, device=DEV)
                ops.moe_combine(y, pos, wts, None, None, one, False)
                ops.moe_combine(parts, pos, wts, None, None, two, False)
                assert (one - two).abs().max() < 1e-4 * float(one.abs().max())
    for a, b in zip(got[128], got[256]):
        assert (a - b).abs().max() <= 1e-2 * float(b.abs().max())
    # one group's rows against the product written out
    order = torch.argsort(ids[:, 0].to(DEV), stable=True)
    rows = order[sizes[1] + sizes[2]:sizes[1] + sizes[2] + sizes[3]]
    want = h[rows].float() @ up[3 * ff:4 * ff].float().t()
    assert (got[256][1][258:258 + 900] - want).abs().max() < 1e-2 * float(want.abs().max())


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("ff, limit", [(12, 0.7), (30, 2.0), (7, 1.5)])
def test_clamped_units_with_weights(ff, limit, dtype):
    from glassbox_amd import ops
    torch.manual_seed(ff)
    E, n = 5, 37
    gu = (torch.randn(n, 2 * E * ff, dtype=F64) * 2).float().to(F64)
    combine = torch.rand(n, E, dtype=F64).float().to(F64)
    combine[:, 1] = 0.0
    act = torch.empty(n, E * ff, dtype=dtype, device=DEV)
    ops.moe_gated_units(_dev(gu), _dev(combine), act, E, ff, (limit, 1.702, 1.0))
    g, u = gu[:, :E * ff].clamp(max=limit), gu[:, E * ff:].clamp(-limit, limit)
    want = g * torch.sigmoid(1.702 * g) * (u + 1) * combine.repeat_interleave(ff, 1)
    tol = 1e-6 if dtype == torch.float32 else 1e-2
    assert (act.cpu().to(F64) - want).abs().max() < tol * float(want.abs().max())
    assert float(act[:, ff:2 * ff].abs().max()) == 0.0


@pytest.mark.parametrize("d, E, top, ff, sizes", [(64, 8, 2, 16, (5, 300)), (128, 4, 2, 64, (3, 2100)), (96, 12, 3, 40, (17, 65, 700)),
                                                  (256, 2, 1, 128, (1100,)), (128, 4, 2, 4096, (2048,))])
def test_experts_on_their_own_tokens_against_every_expert_on_every_token(d, E, top, ff, sizes):
    """The two ways through a step of the routed feed-forward (few rows: every expert on every token, zeros for the ones
    not chosen; many rows: sorted by expert) against the plain sum, with one expert's down matrix a hundred times the
    others', so that a token sent to a wrong expert or weighted wrongly shows."""
    from glassbox_amd.engine.context import Workspace
    from glassbox_amd.parts.moe import RoutedExperts
    torch.manual_seed(d + E)
    limit = 1.5
    part = RoutedExperts(d, E, top, ff, correction=False, scoring="chosen", bias=True, unit="clamped", limit=limit)
    w = {n: torch.randn(s.shape, dtype=F64) * (0.15 if len(s.shape) == 2 else 1.0) for n, s in part.tensor_specs().items()}
    w["router"] = w["router"] * 4
    w["e1.down"] = w["e1.down"] * 100
    w = {n: t.to(torch.bfloat16).to(F64) if t.dim() == 2 else t for n, t in w.items()}
    part.load({n: _dev(t, torch.bfloat16 if t.dim() == 2 else torch.float32) for n, t in w.items()})
    mlp = {"expert": {"ff": ff, "limit": limit}, "router": {"experts": E, "top": top}}
    named = {"m." + k: v for k, v in w.items()}
    ws = Workspace(torch.device(DEV))
    for n in sizes:
        h = torch.randn(n, d, dtype=F64).to(torch.bfloat16).to(F64)
        margins: list = []
        want = pz.experts(named, "m.", mlp, h, rnd=pz.bf16, margins=margins)
        ctx = SimpleNamespace(dtype=torch.bfloat16, buffer=ws.buffer, tuned=True, fuse_norms=True)
        y = torch.full((n, d), 5.0, device=DEV)
        assert part.routed(ctx, n) == (n > 64 and n * top + 64 * E < n * E) == part.adds_in_place(ctx, n)
        made, slices = part.forward(ctx, _dev(h, torch.bfloat16), y, store=True) or (y, 1)
        got = (made if slices == 1 else made[:slices * y.numel()].view(slices, n, d).sum(0)).clone()
        err = (got.cpu().to(F64) - want).abs().max(1).values
        err[margins[0] < 1e-4] = 0.0
        assert float(err.max()) < 2e-2 * float(want.abs().max()), (n, float(err.max()), float(want.abs().max()))
        add = torch.ones(n, d, device=DEV)
        part.forward(ctx, _dev(h, torch.bfloat16), add)
        assert (add - 1.0 - got).abs().max() < 1e-3 * float(want.abs().max())


# ------------------------------------------------------------------------------------------ whole models
REQUESTS = {"a": 150, "b": 77, "c": 41, "d": 3, "e": 1, "f": 97}


def _requests(vocab: int, seed: int = 0):
    return {r: helpers.random_tokens(vocab, n, seed=seed + n) for r, n in REQUESTS.items()}


_ORACLE: dict = {}


def _want(folder: str, tokens, dtype: str) -> np.ndarray:
    key = (folder, tuple(tokens), dtype)
    if key not in _ORACLE:
        cfg, w = pz.load_folder(folder)
        _ORACLE[key] = pz.forward(cfg, rounded(w) if dtype == "bfloat16" else w, list(tokens)).numpy()
    return _ORACLE[key]


def _rounding(folder: str, tokens):
    """How far rounding the activations to bfloat16 moves each position's logits in the plain implementation (root mean
    square over the vocabulary), and the positions at which some router's choice hangs on less than such rounding moves
    its margin by: there an engine that rounds may send the token to other experts than the plain implementation does,
    both being right, and such positions, and those whose convolutions read them directly, are left out of the
    comparison in bfloat16."""
    key = (folder, tuple(tokens), "rounding")
    if key not in _ORACLE:
        cfg, w = pz.load_folder(folder)
        fine, coarse = [], []
        want = pz.forward(cfg, rounded(w), list(tokens), margins=fine)
        moved = pz.forward(cfg, rounded(w), list(tokens), margins=coarse, coarse=True)
        a, b = torch.stack(fine).clamp(max=5.0), torch.stack(coarse).clamp(max=5.0)
        # (one sample of rounding may leave a margin alone by chance: it counts as at least the router's median)
        off = (a - b).abs()
        off = torch.maximum(off, off.median(1, keepdim=True).values)
        close = (a < torch.clamp(ROUTE_TIMES * off, min=ROUTE_MARGIN)).any(0).numpy()
        for back in range(1, (cfg.get("canon") or {"taps": 1})["taps"]):
            close[back:] |= close[:-back].copy()
        _ORACLE[key] = (torch.sqrt(((moved - want) ** 2).mean(1)).numpy(), close)
    return _ORACLE[key]


ROUTE_MARGIN, ROUTE_TIMES = 5e-3, 3.0

#: A 32-bit engine is held to helpers.TOL_F32 of the request's largest logit at every position.  A bfloat16 engine is
#: compared with the plain implementation on the weights it holds by the root mean square of a position's logit
#: differences: at most 3 times what rounding the activations moves that position in the plain implementation itself (at
#: least the median over its request: one sample of rounding is no sharp bound on another), or 1 % of the request's
#: logits' root mean square where that is more; no position may be beyond one and a half times its limit, and one in
#: fifty beyond the limit itself.
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
        moved, close = _rounding(folder, toks)
        lim = np.maximum(BF16_TIMES * np.maximum(moved, np.median(moved)), BF16_FLOOR * float(np.sqrt((want ** 2).mean())))
        assert close.sum() <= max(3, len(toks) // 2), f"{close.sum()} of {len(toks)} positions are close calls of a router"
        err = np.where(close, 0.0, err)
        # a token that went to other experts has other latents in the layers after: the positions behind it that read
        # them are moved too, by less; they get three times the room
        lim = np.where(np.cumsum(close) > 0, 3.0 * lim, lim)
        over = np.nonzero(err > lim)[0]
        assert over.size <= max(1, len(toks) // 50) and float((err / lim).max()) <= 1.5, (
            f"{what}, {dtype}, request {r} ({len(toks)} tokens): position {over[0]} is {err[over[0]]:.3e} off "
            f"(limit {lim[over[0]]:.3e}); {over.size} positions over their limits, worst ratio {(err / lim).max():.2f}")


def _poison(engine) -> None:
    """Garbage in every page and state slot: whatever a request reads, it must have written itself."""
    for lc in engine.layers:
        for t in (lc.k_pages, lc.v_pages, lc.state):
            if t is not None:
                t.fill_(300.0)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", list(CASES))
def test_every_way_of_cutting_requests_into_steps(model_dirs, name, dtype):
    from glassbox_amd.engine import Engine
    folder = folder_of(model_dirs.base, name)
    requests = _requests(CASES[name]["vocab"])
    mixed, peak = helpers.schedule_mixed(requests, seed=3, live=3, tail=20)
    eng = Engine(folder, dtype=dtype, max_tokens=max(peak, 192), max_seqs=3)
    assert all(lc.v_pages is None for lc in eng.layers)
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
    """A prompt of 700 tokens: experts on their own tokens, and contexts of several chunks."""
    from glassbox_amd.engine import Engine
    folder = folder_of(model_dirs.base, name)
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
    """250 tokens one by one after a prompt of four (pages and chunks end many times over; in bfloat16 the steps are
    replayed from graphs), and with plain kernels; the same bits with other pages."""
    from glassbox_amd.engine import Engine
    folder = folder_of(model_dirs.base, "F")
    toks = helpers.random_tokens(97, 254, seed=11)
    steps = helpers.schedule_tail({"x": toks}, 250)
    eng = Engine(folder, dtype=dtype, max_tokens=640, max_seqs=2)
    _poison(eng)
    got = helpers.replay(eng, steps)
    if dtype == "bfloat16":
        assert eng.decode_graphs is not None and eng.decode_graphs.replays > 200
    _check(got, folder, {"x": toks}, dtype, "long decoding")
    eng.step([("first", toks[:37], [])])      # holds the pages and the slot that x had
    again = helpers.replay(eng, steps)
    assert np.array_equal(got["x"], again["x"])
    plain = Engine(folder, dtype=dtype, max_tokens=320, max_seqs=2, graph_decode=False, kernels="plain")
    again = helpers.replay(plain, steps)
    _check(again, folder, {"x": toks}, dtype, "long decoding, plain kernels")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["E", "F"])
def test_layers_of_a_kind_are_made_again_from_the_launches_of_the_first(model_dirs, name, dtype):
    """Layers of one kind, each with a residual buffer of its own: one is recorded, the others are its launches with their
    own tensors, pages, state and residual; the same bits as with every layer walked."""
    from glassbox_amd import ops
    from glassbox_amd.engine import Engine
    folder = folder_of(model_dirs.base, name)
    requests = {"a": helpers.random_tokens(97, 150, seed=1), "b": helpers.random_tokens(97, 41, seed=2)}
    steps = helpers.schedule_whole(requests) + helpers.schedule_chunks(requests, (70, 3, 40)) + helpers.schedule_tail(requests, 5)
    before = ops.TAPE_COUNTS["replayed_layers"]
    taped = helpers.replay(Engine(folder, dtype=dtype, max_tokens=512, max_seqs=2, graph_decode=False), steps)
    assert ops.TAPE_COUNTS["replayed_layers"] >= before + 3 * len(steps)
    before = ops.TAPE_COUNTS["replayed_layers"]
    walked = helpers.replay(Engine(folder, dtype=dtype, max_tokens=512, max_seqs=2, layer_tapes=False, graph_decode=False), steps)
    assert ops.TAPE_COUNTS["replayed_layers"] == before
    assert all(np.array_equal(taped[r], walked[r]) for r in requests)


def test_slots_and_pages_that_are_used_again(model_dirs):
    """Two slots, six requests one after the other in pairs: a request finds the slot (the convolutions' last rows) and the
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


def test_requests_with_a_common_beginning_share_its_pages_where_nothing_else_is_kept(model_dirs):
    """Without a convolution a request leaves nothing but latents: the pages of a common beginning are shared, copied when
    one of two goes its own way, and the logits are those of a request alone."""
    from glassbox_amd.engine import Engine
    folder = folder_of(model_dirs.base, "E")
    first = helpers.random_tokens(97, 60, seed=5)
    second = first[:50] + helpers.random_tokens(97, 20, seed=6)
    eng = Engine(folder, dtype="float32", max_tokens=512, max_seqs=3, prefix_caching=True)
    got = helpers.replay(eng, [{"entries": [("a", first, list(range(60)))], "end": []}])
    reused = eng.add_request("b", second)
    assert reused == 48
    rest = eng.step([("b", second[reused:], list(range(70 - reused)))]).cpu().numpy()
    assert np.abs(rest - _want(folder, second, "float32")[reused:]).max() < helpers.TOL_F32 * max(1.0, float(np.abs(rest).max()))
    eng.fork_request("a", "c")
    ends = [7, 12]
    out = eng.step([("a", [ends[0]], [0]), ("c", [ends[1]], [0])]).cpu().numpy()
    for row, t in zip(out, ends):
        want = _want(folder, first + [t], "float32")[-1]
        assert np.abs(row - want).max() < helpers.TOL_F32 * max(1.0, float(np.abs(want).max()))
    _check(got, folder, {"a": first}, "float32", "shared pages")


# ------------------------------------------------------------------------------------------ generation
def _greedy(cfg, w, prompt, n):
    toks = list(prompt)
    for _ in range(n):
        toks.append(int(torch.argmax(pz.forward(cfg, w, toks)[-1])))
    return toks[len(prompt):]


@pytest.mark.parametrize("name", ["A", "F"])
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
    assert np.abs(np.fromfile(tmp_path / "o" / "0.f32", dtype="<f4").reshape(2, -1) - want[[1, 3]]).max() < 1e-4 * max(1.0, np.abs(want).max())
    assert np.abs(np.fromfile(tmp_path / "o" / "1.f32", dtype="<f4") - want[4]).max() < 1e-4 * max(1.0, np.abs(want).max())
