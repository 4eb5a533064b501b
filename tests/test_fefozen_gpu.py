"""Fefozen on the GPU against the plain implementation: each new or extended kernel alone, then the engine on small
models in float32 and bfloat16: every layer, whole prompts, decoding through state and cache, portions down to two tokens,
unequal batches with slots and pages used again, first tokens, keys far back and at page borders, portions at the edges of
the recurrence's chunks, long decoding, greedy generation through ``Engine``, the replay loop and a named size."""
import copy
import json
import os

import numpy as np
import pytest
import torch

import plain_fefozen as plain
import tiny_fefozen as tiny
from test_pupalix_gpu import _paged
from test_zimorax_gpu import DEV, DTYPES, F64, check, dev, items_ctx, make_runner, rounded, run_schedule

pytestmark = pytest.mark.gpu


def _i32(values):
    return torch.tensor(list(values), dtype=torch.int32, device=DEV)


def _delta_ctx(lens, slots, starts, padding=0):
    """(token_item, positions, item_len, item_tok_off, item_slot), with ``padding`` rows of no item behind."""
    ti, il, off, sl = items_ctx(lens, slots)
    pos = [s + p for s, n in zip(starts, lens) for p in range(n)]
    return torch.cat([ti, _i32([-1] * padding)]), _i32(pos + [-1] * padding), il, off, sl


# ------------------------------------------------------------------ kernels alone
@pytest.mark.parametrize("dtype", list(DTYPES))
@pytest.mark.parametrize("T,W", [(5, 64), (3, 90), (9, 2048), (2, 4096), (4, 2050), (1, 7168), (3, 9000), (2, 8), (300, 320)])
def test_a_branch_through_a_norm_into_the_stream_and_the_next_norm(dtype, T, W):
    from swifttransformer_amd.ops import kernels as K
    g = torch.Generator().manual_seed(T * 10 + W)
    dt = DTYPES[dtype]
    y = torch.randn(T, W, generator=g, dtype=F64) * torch.linspace(0.01, 4.0, W, dtype=F64)
    x = torch.randn(T, W, generator=g, dtype=F64) * 2.0
    a, b = 0.3 * torch.randn(W, generator=g, dtype=F64), 0.3 * torch.randn(W, generator=g, dtype=F64)
    want = x + plain.shifted_rms(y, a, 1e-5)
    got = K.rms_onto(dev(y), dev(x), dev(1.0 + a), 1e-5)
    check(got, want.numpy(), torch.float32, "the stream")
    got, h = K.rms_onto(dev(y), dev(x), dev(1.0 + a), 1e-5, (dev(1.0 + b), 1e-3), dt)
    check(got, want.numpy(), torch.float32, "the stream beside the next norm")
    check(h, plain.shifted_rms(want, b, 1e-3).numpy(), dt, "the next norm")


def _latent_layout(rank, r):
    off = -(-rank // 8) * 8 if r else rank
    return off, -(-(off + r) // 16) * 16, -(-rank // 16) * 16


@pytest.mark.parametrize("dtype", list(DTYPES))
@pytest.mark.parametrize("q_rank,rank,r,dims,ps", [(40, 32, 8, 8, 4), (37, 21, 6, 6, 2), (64, 130, 64, 24, 16), (16, 16, 0, 0, 8),
                                                   (300, 512, 64, 64, 16), (1600, 270, 16, 16, 12)])
def test_query_latent_and_cache_entries_from_one_products_rows(dtype, q_rank, rank, r, dims, ps):
    """Two portions of two requests over shuffled pages, a padding row; entries whole (zeros between and behind the parts),
    pages of nobody untouched; without a cache the query latent alone."""
    from swifttransformer_amd.ops import kernels as K
    from swifttransformer_amd.parts.position import rotary_frequencies
    g = torch.Generator().manual_seed(q_rank + rank)
    dt, eps, base = DTYPES[dtype], 1e-4, 90.0
    off, entry, _ = _latent_layout(rank, r)
    lens = [21, 9]
    bt, pages = _paged(lens, ps, g)
    cache = torch.full((pages, 1, ps, entry), 9.0, dtype=dt, device=DEV)
    gq, gc = 1.0 + 0.3 * torch.randn(q_rank, generator=g), 1.0 + 0.3 * torch.randn(rank, generator=g)
    freq = dev(torch.tensor(rotary_frequencies(dims, base)[0])) if r else None
    width = q_rank + rank + r + 5
    rows = [torch.randn(n, width, generator=g) * 2.0 for n in lens]
    used = set()
    for a, e in ((0, 4), (4, 99)):
        x = torch.cat([t[a:e] for t in rows] + [torch.full((1, width), float("nan"))])
        pos = _i32([p for t in rows for p in range(t.shape[0])[a:e]] + [-1])
        item = _i32([b for b, t in enumerate(rows) for _ in range(t.shape[0])[a:e]] + [-1])
        cq = K.latent_inputs(dev(x), q_rank, q_rank + 3, dev(gq), eps, cache, dtype=dt, gain=dev(gc), rank=rank, tail_off=off, tail=r,
                             tail_freq=freq, ctx_arrays=(item, pos, bt.to(DEV)))[:-1]
        x64 = x[:-1].to(F64)
        check(cq[:, :q_rank], (plain.unit_rms(x64[:, :q_rank], eps) * gq.to(F64)).numpy(), dt, "query latent")
        assert float(cq[:, q_rank:].abs().sum()) == 0.0
        alone = K.latent_inputs(dev(x[:-1]), q_rank, q_rank, dev(gq), eps, dtype=dt)
        assert torch.equal(alone, cq[:, :q_rank])
    for b, t in enumerate(rows):
        n = t.shape[0]
        at = [(int(bt[b, p // ps]), p % ps) for p in range(n)]
        used |= {page for page, _ in at}
        got = torch.stack([cache[page, 0, s] for page, s in at])
        x64 = t.to(F64)
        c = plain.unit_rms(x64[:, q_rank:q_rank + rank], eps) * gc.to(F64)
        check(got[:, :rank], c.numpy(), dt, f"latents of request {b}")
        if r:
            tail = plain.turn(x64[:, q_rank + rank:q_rank + rank + r], dims, base, True)
            check(got[:, off:off + r], tail.numpy(), dt, f"turned parts of request {b}")
        blank = torch.ones(entry, dtype=torch.bool)
        blank[:rank] = False
        blank[off:off + r] = False
        assert float(got[:, blank.to(DEV)].abs().sum()) == 0.0
    for page in range(pages):
        if page not in used:
            assert (cache[page] == 9.0).all()


def _latent_reference(q, entries, H, rank, off, r, dims, base, scale, sink, window):
    """q [T, H, entry] before the turn, entries [T, entry], float64 -> [T, H, rank]."""
    T = q.shape[0]
    q = q.clone()
    if r:
        q[..., off:off + r] = plain.turn(q[..., off:off + r], dims, base, True)
    s = torch.matmul(q.transpose(0, 1), entries.T) * scale
    i, j = torch.arange(T)[:, None], torch.arange(T)[None, :]
    seen = (j <= i) & ((i - j < window) if window else True)
    p = plain.softmax_with_sink(s.masked_fill(~seen[None], float("-inf")), sink)
    return torch.matmul(p, entries[:, :rank]).transpose(0, 1)


@pytest.mark.parametrize("dtype", list(DTYPES))
@pytest.mark.parametrize("H,rank,r,dims,ps,sinks,scale,window", [
    (4, 32, 8, 8, 4, True, 0.3, 0), (3, 21, 6, 6, 2, False, 0.4, 0), (20, 130, 64, 24, 16, True, 0.2, 0), (1, 16, 0, 0, 8, False, 0.7, 0),
    (40, 270, 16, 16, 12, True, 0.2, 0), (32, 128, 32, 32, 16, False, 0.15, 0), (16, 160, 32, 32, 16, True, 0.15, 33),
    (7, 512, 64, 64, 16, True, 0.1, 0), (5, 224, 32, 32, 16, True, -0.15, 0), (2, 64, 64, 64, 3, False, 0.2, 65), (33, 96, 0, 0, 16, True, 0.2, 1)])
def test_attention_over_a_latent_cache_by_tiles_and_by_rows(dtype, H, rank, r, dims, ps, sinks, scale, window):
    """Requests of several lengths over shuffled pages whose other entries are not numbers, one stronger key far back: tiles
    (whole items, a late portion, a padding tile), rows with 1, 3 and 40 shares of the keys and picked rows, and the
    product a head behind either, gated and not."""
    from swifttransformer_amd.engine.batch import StepItem
    from swifttransformer_amd.ops import kernels as K
    from swifttransformer_amd.parts.attention import plan_tiles
    from swifttransformer_amd.parts.position import rotary_frequencies
    g = torch.Generator().manual_seed(H * 100 + rank)
    dt, base, vd = DTYPES[dtype], 70.0, 12 if H != 3 else 7
    off, entry, od = _latent_layout(rank, r)
    lens = [150, 3, 67, 1]
    bt, pages = _paged(lens, ps, g)
    cache = torch.full((pages, 1, ps, entry), float("nan"), dtype=dt, device=DEV)
    sink = torch.randn(H, generator=g) * 1.5 if sinks else None
    freq = dev(torch.tensor(rotary_frequencies(dims, base)[0])) if r else None
    sh = K.LatentShape(H, entry, od, scale, off, freq, 1.0, dev(sink) if sinks else None, window)
    qs, refs = [], []
    for b, n in enumerate(lens):
        e = torch.zeros(n, entry)
        e[:, :rank] = torch.randn(n, rank, generator=g)
        if r:
            e[:, off:off + r] = torch.randn(n, r, generator=g)
        if n > 20:
            e[n // 7] *= 2.0                                              # a key that stands out
        q = torch.randn(n, H, entry, generator=g)
        e, q = rounded(e, dtype), rounded(q, dtype)
        for p in range(n):
            cache[int(bt[b, p // ps]), 0, p % ps] = dev(e[p], dt)
        refs.append(_latent_reference(q, e, H, rank, off, r, dims, base, scale, sink.to(F64) if sinks else None, window))
        qs.append(q)
    q_all, ref = dev(torch.cat(qs).reshape(-1, H * entry), dt), torch.cat(refs)
    flat = ref.reshape(-1, H * rank).numpy()
    cut = lambda o: o.view(-1, H, od)[:, :, :rank].reshape(-1, H * rank)
    ti, pos = _i32([b for b, n in enumerate(lens) for _ in range(n)]), _i32([p for n in lens for p in range(n)])
    btd = bt.to(DEV)
    loosen = 2.0
    w = rounded(torch.randn(H, vd, rank, generator=g) / rank ** 0.5, dtype)
    wd = torch.nn.functional.pad(dev(w, dt), (0, od - rank)).contiguous()
    z = torch.randn(ref.shape[0], H * vd + 3, generator=g)
    gate = dev(z)[:, 1:1 + H * vd]
    up = torch.einsum("thr,hvr->thv", ref, w).reshape(-1, H * vd)
    gated = (up * torch.sigmoid(z[:, 1:1 + H * vd].to(F64))).numpy()
    # rows
    for splits in (1, 3, 40):
        part = K.latent_rows(q_all, cache, ti, pos, btd, sh, splits)
        out = torch.full((q_all.shape[0], H * od), 3.0, dtype=dt, device=DEV)
        K.latent_merge(part, out)
        check(cut(out), flat, dt, f"rows, {splits} shares", loosen)
        check(K.latent_up(part, wd, gate, ti), gated, dt, f"rows, {splits} shares, product and gate", loosen)
    check(K.latent_up(part, wd, None, ti), up.numpy(), dt, "product without a gate", loosen)
    ids = _i32([151, 5, -1, 219])
    part = K.latent_rows(q_all, cache, ti, pos, btd, sh, 2, ids)
    out = torch.full((q_all.shape[0], H * od), 3.0, dtype=dt, device=DEV)
    K.latent_merge(part, out, ids)
    check(cut(out)[[151, 5, 219]], flat[[151, 5, 219]], dt, "picked rows", loosen)
    assert (out[[0, 1, 150, 220]] == 3.0).all()
    # padding rows of a batch
    item = ti.clone()
    item[7] = -1
    y = K.latent_up(K.latent_rows(q_all, cache, item, pos, btd, sh, 2), wd, gate, item)
    keep = [t for t in range(ref.shape[0]) if t != 7]
    check(y[keep], gated[keep], dt, "beside a padding row", loosen)
    # tiles: whole items, then a late portion of the first (its queries alone)
    items = [StepItem(slot=b, start=0, tokens=[0] * n) for b, n in enumerate(lens)]
    for bucketed in (False, True):
        plan = plan_tiles(items, 1, 64, bucketed=bucketed)
        out = torch.full((q_all.shape[0], H * od), 3.0, dtype=dt, device=DEV)
        offs = np.concatenate([[0], np.cumsum(lens)[:-1]])
        tile_item, tile_q0 = np.append(plan.arrays["tile_item"], -1), np.append(plan.arrays["tile_q0"], 0)
        K.latent_tiles(q_all, cache, _i32(tile_item), _i32(tile_q0), _i32(offs), _i32([0] * 4), _i32(lens), btd, sh, out)
        check(cut(out), flat, dt, "tiles", loosen)
    check(K.latent_up(out, wd, gate), gated, dt, "tiles, product and gate", loosen)
    check(K.latent_up(out, wd), up.numpy(), dt, "tiles, product without a gate", loosen)
    n = 150 - 79
    out = torch.full((n, H * od), 3.0, dtype=dt, device=DEV)
    K.latent_tiles(q_all[79:150].contiguous(), cache, _i32([0, 0]), _i32([0, 64]), _i32([0]), _i32([79]), _i32([n]), btd, sh, out)
    check(cut(out), flat[79:150], dt, "a late portion", loosen)


def _delta_plain(x, w, H, G, dk, dv, gain, eps, unit_eps=1e-6):
    """The mixer between its two products on rows x = q | k | v | gate | strength | decay of one sequence."""
    T = x.shape[0]
    k0, v0, z0 = G * dk, 2 * G * dk, 2 * G * dk + H * dv
    q, k, v = (plain.short_filter(x[:, a:b], w["conv"][a:b]) for a, b in ((0, k0), (k0, v0), (v0, z0)))
    unit = lambda t: t / torch.sqrt((t * t).sum(-1, keepdim=True) + unit_eps)
    q = unit(q.view(T, G, dk)).repeat_interleave(H // G, dim=1) * dk ** -0.5
    k = unit(k.view(T, G, dk)).repeat_interleave(H // G, dim=1)
    z, b, a = x[:, z0:z0 + H * dv].view(T, H, dv), x[:, z0 + H * dv:z0 + H * dv + H], x[:, z0 + H * dv + H:z0 + H * dv + 2 * H]
    g = torch.exp(-torch.exp(w["A_log"]) * torch.nn.functional.softplus(a + w["dt_bias"]))
    o = plain.delta_memory(q, k, v.view(T, H, dv), torch.sigmoid(b), g)
    return (plain.unit_rms(o, eps) * gain * z * torch.sigmoid(z)).reshape(T, H * dv)


@pytest.mark.parametrize("dtype", list(DTYPES))
@pytest.mark.parametrize("H,G,dk,dv,taps", [(4, 2, 12, 20, 4), (3, 3, 5, 7, 5), (3, 1, 72, 40, 1), (2, 2, 16, 64, 3), (1, 1, 32, 32, 2),
                                            (2, 1, 8, 130, 2), (4, 1, 64, 64, 4), (2, 2, 128, 128, 4), (1, 1, 256, 256, 8), (2, 1, 255, 33, 6)])
def test_the_delta_rule_whole_token_by_token_and_in_portions(dtype, H, G, dk, dv, taps):
    """Two requests of unequal length in their slots beside others': whole, one token at a time, and portions cut at and off the
    chunks' edges, with a padding row that is not a number; slots of others stay as they are."""
    from swifttransformer_amd.ops import kernels as K
    g = torch.Generator().manual_seed(H * 1000 + dk + dv)
    dt, eps = DTYPES[dtype], 1e-4
    C, width = 2 * G * dk + H * dv, K.delta_row(H, G, dk, dv)
    w = {"conv": torch.cat([0.4 * torch.randn(C, taps - 1, generator=g), 1.0 + 0.2 * torch.randn(C, 1, generator=g)], 1).to(F64),
         "A_log": (torch.randn(H, generator=g) - 1.5).to(F64), "dt_bias": torch.randn(H, generator=g).to(F64)}
    gain = (1.0 + 0.3 * torch.randn(dv, generator=g)).to(F64)
    lens = {4: 150, 1: 21} if dk < 200 else {4: 90, 1: 7}
    seqs = {}
    for s, n in lens.items():
        x = torch.randn(n, width + 2, generator=g) * 1.5
        x[:, G * dk:2 * G * dk] = 0.8 * x[:, :G * dk] + 0.6 * x[:, G * dk:2 * G * dk]     # keys that lean to the queries
        seqs[s] = x
    want = {s: _delta_plain(x.to(F64), w, H, G, dk, dv, gain, eps) for s, x in seqs.items()}
    taps_w = dev(w["conv"].T)
    n4 = lens[4]
    schedules = {"whole": [[(4, n4), (1, lens[1])]],
                 "token by token": [[(1, 1), (4, 1)]] * lens[1] + [[(4, 1)]] * (n4 - lens[1]),
                 "portions": [[(4, 2), (1, 1)], [(1, 2), (4, 1)], [(4, 61)], [(4, 1), (1, 1)], [(1, 3), (4, 2)], [(4, n4 - 67)]]}
    for what, steps in schedules.items():
        state = torch.full((6, K.delta_slot(H, G, dk, dv, taps)), 5.5, device=DEV)
        state[[4, 1]] = 0.0                                     # what admission leaves
        done = {4: 0, 1: 0}
        for step in steps:
            cl, slots, starts = [n for _, n in step], [s for s, _ in step], [done[s] for s, _ in step]
            single = all(n == 1 for n in cl)
            pad = 0 if single else 1
            x = torch.cat([seqs[s][done[s]:done[s] + n] for s, n in step] + [torch.full((pad, width + 2), float("nan"))])
            got = K.delta_rule(dev(x), taps_w, dev(w["A_log"]), dev(w["dt_bias"]), dev(gain), state, _delta_ctx(cl, slots, starts, pad),
                               H, G, dk, dv, eps, 1e-6, dt, all_single=single)
            ref = torch.cat([want[s][done[s]:done[s] + n] for s, n in step])
            check(got[:ref.shape[0]], ref.numpy(), dt, f"{what} {step}", loosen=4.0 if dtype == "float32" else 1.0)
            for s, n in step:
                done[s] += n
        assert (state[[0, 2, 3, 5]] == 5.5).all()


@pytest.mark.parametrize("dtype", ["float32"])
def test_delta_rule_with_decays_and_strengths_at_their_ends(dtype):
    """Decays next to zero (a chunk's products of them would vanish or overflow where they were divided by), next to one, and
    strengths next to one and zero, in one chunk and across chunks."""
    from swifttransformer_amd.ops import kernels as K
    g = torch.Generator().manual_seed(3)
    H, G, dk, dv, T, eps = 4, 2, 16, 16, 200, 1e-3
    C, width = 2 * G * dk + H * dv, K.delta_row(H, G, dk, dv)
    w = {"conv": torch.ones(C, 1, dtype=F64), "A_log": torch.tensor([3.0, -6.0, 1.0, 0.0], dtype=F64), "dt_bias": torch.tensor([2.0, -3.0, 0.0, 30.0], dtype=F64)}
    x = torch.randn(T, width, generator=g)
    x[:, G * dk:2 * G * dk] = 0.9 * x[:, :G * dk] + 0.3 * x[:, G * dk:2 * G * dk]
    x[:, C + H * dv:C + H * dv + H] = torch.tensor([8.0, 8.0, -8.0, 0.0])
    x[:, C + H * dv + H:] = torch.randn(T, H, generator=g) * 10.0
    gain = torch.ones(dv, dtype=F64)
    want = _delta_plain(x.to(F64), w, H, G, dk, dv, gain, eps)
    for cuts in ([T], [64, 64, 72], [1] * T, [63, 2, 135]):
        state = torch.zeros((1, K.delta_slot(H, G, dk, dv, 1)), device=DEV)
        at, outs = 0, []
        for c in cuts:
            outs.append(K.delta_rule(dev(x)[at:at + c], dev(w["conv"].T), dev(w["A_log"]), dev(w["dt_bias"]), dev(gain), state,
                                     _delta_ctx([c], [0], [at]), H, G, dk, dv, eps, 1e-6, torch.float32, all_single=c == 1))
            at += c
        check(torch.cat(outs), want.numpy(), torch.float32, f"{cuts[:3]}", loosen=6.0)


@pytest.mark.parametrize("dtype", list(DTYPES))
@pytest.mark.parametrize("E,I,top,W,F,T,limit", [(6, 2, 2, 64, 24, 37, 1.0), (4, 1, 5, 90, 20, 9, 0.6), (8, 0, 1, 128, 40, 300, 2.0),
                                                 (2, 3, 3, 48, 16, 150, 1.2), (8, 4, 2, 256, 192, 420, 0.8), (70, 10, 4, 64, 16, 21, 1.5),
                                                 (12, 2, 4, 72, 136, 330, 1.0), (3, 2, 1, 64, 16, 40, 1.0)])
def test_clamped_experts_and_identity_experts_chosen_by_corrected_shares(dtype, E, I, top, W, F, T, limit):
    from swifttransformer_amd.ops import kernels as K
    g = torch.Generator().manual_seed(E * 10 + top)
    dt, n = DTYPES[dtype], E + I
    x = rounded(torch.randn(T, W, generator=g) * 1.5, dtype)
    gate, up = (rounded(torch.randn(E, F, W, generator=g) * 1.5 / W ** 0.5, dtype) for _ in range(2))
    down = rounded(torch.randn(E, W, F, generator=g) / F ** 0.5, dtype)
    # logits a permutation of well separated levels a row (no close call), two of them moved by corrections of another order
    levels = torch.linspace(-2.0, 2.0, n, dtype=F64)
    logits = torch.stack([levels[torch.randperm(n, generator=g)] for _ in range(T)]).to(torch.float32)
    correction = torch.zeros(n)
    correction[n // 2], correction[0] = 2.0, -2.0
    ref = torch.zeros(T, W, dtype=F64)
    for t in range(T):
        for e, s in plain.route(logits[t].to(F64), correction.to(F64), top):
            ref[t] += s * (x[t] if e >= E else plain.expert(x[t], gate[e], up[e], down[e], limit))
    item = torch.zeros(T, dtype=torch.int32)
    item[T // 2] = -1                                           # a padding row
    ref[T // 2] = 0.0
    kw = dict(top=top, limit=limit, token_item=item.to(DEV), style="softmax_corrected", correction=dev(correction), identity=I, clamped=True)
    wide = torch.cat([dev(logits), torch.full((T, 5), 99.0, device=DEV)], dim=1)      # rows longer than the outputs
    for z in (dev(logits), wide):
        got = K.routed_experts(dev(x, dt), z, dev(gate, dt), dev(up, dt), dev(down, dt), None, **kw)
        check(got, ref.numpy(), dt, "the sum alone", loosen=2.0)
    base = torch.randn(T, W, generator=g)
    got = K.routed_experts(dev(x, dt), dev(logits), dev(gate, dt), dev(up, dt), dev(down, dt), dev(base), out_scale=0.6, **kw)
    check(got, (0.6 * ref + base.to(F64)).numpy(), dt, "onto a stream", loosen=2.0)


# ------------------------------------------------------------------ the engine on small models
@pytest.fixture(scope="module")
def models(tmp_path_factory):
    root = tmp_path_factory.mktemp("fefozen")
    out = {}
    for name, cfg in tiny.CONFIGS.items():
        d = tiny.write_folder(cfg, str(root / name), 13)
        out[name] = (d,) + plain.load_folder(d)
    return out


@pytest.mark.parametrize("dtype", list(DTYPES))
@pytest.mark.parametrize("name", list(tiny.CONFIGS))
def test_every_layer_against_the_plain_residual_stream(models, name, dtype):
    from swifttransformer_amd.engine.batch import pack_batch
    from swifttransformer_amd.engine.step import StepEntry
    folder, cfg, w = models[name]
    seq = tiny.prompt(23, cfg["vocab"], 1)
    want = plain.residual_streams(cfg, w, seq)
    ps = tiny.PAGE_SIZE[name]
    runner = make_runner(folder, dtype, ps, 8 + 23 // ps, record_after=0)
    model = runner.model
    runner.admit(0)
    items = runner.prepare([StepEntry(0, seq, [])])
    ctx = pack_batch(items, runner.paged_group_ids, runner.max_pages_per_seq, ps, DEV, vocab_size=cfg["vocab"],
                     max_positions=model.max_positions, planners=runner.planners)
    seen = []
    for layer in model.layers:
        def fwd(x32, *a, _orig=layer.arrangement.forward, **kw):
            out = _orig(x32, *a, **kw)
            seen.append(out.clone())
            return out
        layer.arrangement.forward = fwd
    model.forward_layers(ctx, runner.cache.views)
    assert len(seen) == want.shape[0] == len(cfg["layers"])
    for i, got in enumerate(seen):
        check(got, want[i].numpy(), DTYPES[dtype], f"{name} {dtype} after layer {i}", loosen=2.0)


@pytest.mark.parametrize("recording", [0, 2])
@pytest.mark.parametrize("dtype", list(DTYPES))
@pytest.mark.parametrize("name", list(tiny.CONFIGS))
def test_whole_decoded_and_in_portions(models, name, dtype, recording):
    folder, cfg, w = models[name]
    seq = tiny.prompt(150, cfg["vocab"], 2)
    ref = plain.logits(cfg, w, seq).numpy()
    ps = tiny.PAGE_SIZE[name]
    runner = make_runner(folder, dtype, ps, -(-150 // ps) + 2, record_after=recording)
    what = f"{name} {dtype}"
    run_schedule(runner, {0: seq}, {0: ref}, [[(0, 150)]], dtype, what + " whole", loosen=2.0)
    run_schedule(runner, {0: seq}, {0: ref}, [[(0, 90)]] + [[(0, 1)]] * 60, dtype, what + " decoded", loosen=2.0)
    run_schedule(runner, {0: seq[:40]}, {0: ref[:40]}, [[(0, 1)]] * 40, dtype, what + " token by token", loosen=2.0)
    run_schedule(runner, {0: seq}, {0: ref}, [[(0, n)] for n in (11, 2, 13, 64, 3, 2, 40, 15)], dtype, what + " portions", loosen=2.0)
    run_schedule(runner, {0: seq[:80]}, {0: ref[:80]}, [[(0, 2)]] * 40, dtype, what + " two at a time", loosen=2.0)
    assert all(g.pool.num_free == g.pool.num_pages for g in runner.manager.paged_groups)


@pytest.mark.parametrize("dtype", list(DTYPES))
@pytest.mark.parametrize("name", list(tiny.CONFIGS))
def test_first_tokens_and_unequal_batches_with_slots_and_pages_used_again(models, name, dtype):
    folder, cfg, w = models[name]
    lens = {0: 70, 1: 1, 2: 33, 3: 9, 4: 26, 5: 2, 6: 41}
    seqs = {r: tiny.prompt(n, cfg["vocab"], 10 + r) for r, n in lens.items()}
    refs = {r: plain.logits(cfg, w, s).numpy() for r, s in seqs.items()}
    ps = tiny.PAGE_SIZE[name]
    runner = make_runner(folder, dtype, ps, 3 * (-(-70 // ps)) + 4, record_after=2, max_seqs=3)
    schedule = [[(0, 30), (1, 1), (2, 2)],              # a request of one token ends at once: its slot comes back
                [(2, 1), (0, 2), (3, 9)],               # a new request in the freed slot beside portions
                [(0, 1), (2, 30)],                      # request 2 ends
                [(4, 13), (0, 1)], [(0, 36), (4, 1)],   # request 0 ends
                [(5, 1), (4, 12), (6, 3)], [(5, 1), (6, 2)], [(6, 36)]]
    run_schedule(runner, seqs, refs, schedule, dtype, f"{name} {dtype} mixed", loosen=2.0)
    assert runner.manager.num_free_slots == 3
    assert all(g.pool.num_free == g.pool.num_pages for g in runner.manager.paged_groups)


@pytest.mark.parametrize("dtype", list(DTYPES))
def test_portions_at_the_edges_of_the_recurrences_chunks_beside_others(models, dtype):
    folder, cfg, w = models["A"]
    seqs = {0: tiny.prompt(330, cfg["vocab"], 7), 1: tiny.prompt(40, cfg["vocab"], 8)}
    refs = {r: plain.logits(cfg, w, s).numpy() for r, s in seqs.items()}
    ps = tiny.PAGE_SIZE["A"]
    runner = make_runner(folder, dtype, ps, -(-330 // ps) + -(-40 // ps) + 2, record_after=2)
    schedule = [[(0, 63), (1, 20)], [(1, 1), (0, 65)], [(0, 1), (1, 1)], [(1, 2), (0, 64)], [(0, 16), (1, 16)]] + \
               [[(0, 1)]] * 50 + [[(0, 2)], [(0, 69)]]
    run_schedule(runner, seqs, refs, schedule, dtype, f"A {dtype} mixed", loosen=2.0)


def _layers_alone(cfg0, w0, picked, tmp_path, change):
    """A model made of the layers ``picked`` of ``cfg0`` (a lender and its borrower keep their bond), without feed-forwards."""
    cfg = copy.deepcopy(cfg0)
    cfg["layers"] = [dict(cfg["layers"][i], mlp=None) for i in picked]
    w = {k: v.to(torch.float32).clone() for k, v in w0.items() if k in ("embed", "final.norm")}
    for n, i in enumerate(picked):
        m = cfg["layers"][n]["mixer"]
        if m.get("kv_from") is not None:
            m["kv_from"] = picked.index(m["kv_from"])
        pre = f"l{i}."
        w.update({f"l{n}." + k[len(pre):]: v.to(torch.float32).clone() for k, v in w0.items()
                  if k.startswith(pre) and ".mlp." not in k and "norm2" not in k})
        change(m, w, f"l{n}.")
    folder = tiny.write_folder(cfg, str(tmp_path / "alone"), 0, weights=w)
    return (folder,) + plain.load_folder(folder)


@pytest.mark.parametrize("dtype", list(DTYPES))
@pytest.mark.parametrize("name,picked,ps", [("A", [2], 4), ("A", [1, 3], 16), ("C", [1], 8), ("E", [0], 12)])
def test_peaked_attention_far_back_and_at_page_borders(models, tmp_path, dtype, name, picked, ps):
    """Latent attentions alone (one with a sink, and a lender with its borrower), their scores scaled up so that the softmax picks
    single keys: a key that is wrongly seen or missed, or turned by a wrong position, moves the row.  The plain model's own
    parts say which key each query of the last layer weighs most: some far back, some at page borders, some the
    sequence's first."""
    _, cfg0, w0 = models[name]
    # (behind a peaked layer the next one's scores carry its rounding on)
    boost = (30.0 if len(picked) == 1 else 10.0) if dtype == "float32" else 3.0

    def change(m, w, p):
        m["scale"] = m["scale"] * boost
        if p + "mix.sink" in w:
            w[p + "mix.sink"] = w[p + "mix.sink"] * boost           # still one term among equals
    folder, cfg, w = _layers_alone(cfg0, w0, picked, tmp_path, change)
    T = 330
    seq = tiny.prompt(T, cfg["vocab"], 5)
    ref, parts = None, {}
    orig = plain.softmax_with_sink

    def spy(s, sink=None):
        parts["scores"] = s
        return orig(s, sink)
    plain.softmax_with_sink = spy
    try:
        ref = plain.logits(cfg, w, seq).numpy()
    finally:
        plain.softmax_with_sink = orig
    best = [(t, int(row[t].argmax())) for row in parts["scores"] for t in range(T)]
    assert max(t - b for t, b in best) > 150
    assert any(b % ps == 0 for _, b in best) and any(b % ps == ps - 1 for _, b in best)
    assert any(b < 2 and t > 2 for t, b in best)
    runner = make_runner(folder, dtype, ps, -(-T // ps) + 2, record_after=2, max_seqs=2)
    loosen = 4.0
    run_schedule(runner, {0: seq}, {0: ref}, [[(0, T)]], dtype, "whole", loosen)
    run_schedule(runner, {0: seq}, {0: ref}, [[(0, 230)]] + [[(0, 1)]] * 100, dtype, "decoded", loosen)
    run_schedule(runner, {0: seq}, {0: ref}, [[(0, 15)], [(0, 2)], [(0, 111)], [(0, 130)], [(0, 2)], [(0, 70)]], dtype, "portions", loosen)
    assert all(g.pool.num_free == g.pool.num_pages for g in runner.manager.paged_groups)


@pytest.mark.parametrize("dtype", list(DTYPES))
def test_a_sink_that_takes_most_of_the_weight_and_one_that_takes_none(models, tmp_path, dtype):
    """Early rows see few keys, so a large sink halves and more what they read; a sink that was left out, counted twice (once a
    share of the keys) or scaled moves them."""
    _, cfg0, w0 = models["A"]

    def change(m, w, p):
        H = m["heads"]
        w[p + "mix.sink"] = torch.tensor([4.0, -30.0, 2.0, 6.0, 0.0, 8.0][:H])
        m["scale"] = 0.05
    folder, cfg, w = _layers_alone(cfg0, w0, [2], tmp_path, change)
    seqs = {0: tiny.prompt(300, cfg["vocab"], 25), 1: tiny.prompt(30, cfg["vocab"], 26)}
    refs = {r: plain.logits(cfg, w, s).numpy() for r, s in seqs.items()}
    w2 = {**w, "l0.mix.sink": torch.full_like(w["l0.mix.sink"], -40.0)}
    assert np.abs(plain.logits(cfg, w2, seqs[0]).numpy() - refs[0]).max() > 0.2 * refs[0].std()
    runner = make_runner(folder, dtype, 4, 90, record_after=2, max_seqs=2)
    run_schedule(runner, seqs, refs, [[(0, 1), (1, 1)], [(0, 1), (1, 9)], [(0, 7), (1, 1)], [(0, 250), (1, 19)]] + [[(0, 1)]] * 41, dtype, "sinks", 2.0)


@pytest.mark.parametrize("dtype", list(DTYPES))
def test_a_state_that_keeps_a_token_for_long(models, tmp_path, dtype):
    """A delta rule alone that decays next to nothing, its keys all but orthogonal by their tokens' codes: the first tokens still
    show hundreds of tokens later; a state that was lost, cut or mixed with another request's moves every later row."""
    _, cfg0, w0 = models["C"]

    def change(m, w, p):
        w[p + "mix.A_log"] = torch.full_like(w[p + "mix.A_log"], -8.0)
        w[p + "mix.b"] *= 0.3
    folder, cfg, w = _layers_alone(cfg0, w0, [0], tmp_path, change)
    seqs = {0: tiny.prompt(300, cfg["vocab"], 5), 1: tiny.prompt(120, cfg["vocab"], 6)}
    seqs[0][0] = 60                                             # a token of its own at the start, asked for again at the end
    seqs[0][1:299] = [t % 60 for t in seqs[0][1:299]]
    seqs[0][299] = 60
    refs = {r: plain.logits(cfg, w, s).numpy() for r, s in seqs.items()}
    other = plain.logits(cfg, w, [0] + seqs[0][1:]).numpy()
    assert np.abs(other[299] - refs[0][299]).max() > 0.05 * refs[0][299].std()      # the first token shows at the end
    runner = make_runner(folder, dtype, 16, 40, record_after=2, max_seqs=2)
    run_schedule(runner, seqs, refs, [[(0, 40), (1, 2)]] + [[(0, 1), (1, 1)]] * 30 + [[(1, 70), (0, 1)], [(0, 2), (1, 18)], [(0, 150)]] +
                 [[(0, 1)]] * 77, dtype, "beside another", loosen=3.0)


def test_greedy_generation_through_the_engine(models):
    from swifttransformer_amd.engine.engine import Engine
    from swifttransformer_amd.sampling import SamplingParams
    folder, cfg, w = models["A"]
    prompts = [tiny.prompt(n, cfg["vocab"], 40 + i) for i, n in enumerate((1, 7, 19, 30, 4, 12))]
    eng = Engine(folder, dtype="fp32", page_size=4, num_pages=40, max_seqs=3, max_batched_tokens=24, prefill_chunk=10)
    outs = eng.generate(prompts, SamplingParams(max_new_tokens=12, ignore_eos=True))
    for p, o in zip(prompts, outs):
        assert o == plain.generate(cfg, w, p, 12), f"prompt of {len(p)} tokens"
    assert eng.runner.manager.num_free_slots == 3
    # bfloat16: every chosen token is the plain model's best for the engine's own sequence, up to rounding
    eng = Engine(folder, dtype="bf16", page_size=4, num_pages=40, max_seqs=3, max_batched_tokens=24, prefill_chunk=10)
    outs = eng.generate(prompts[:3], SamplingParams(max_new_tokens=8, ignore_eos=True))
    for p, o in zip(prompts, outs):
        logits = plain.logits(cfg, w, list(p) + list(o)).numpy()
        for i, tok in enumerate(o):
            row = logits[len(p) - 1 + i]
            assert row.max() - row[tok] <= 0.05 * row.std() + 0.02 * abs(row.max())


def test_a_request_that_loses_its_pages_starts_again_from_cleared_state(models):
    """A pool that cannot hold the requests together: the scheduler takes pages back from a running request, which is
    computed again later in a slot that held another request's state and filter inputs."""
    from swifttransformer_amd.engine.engine import Engine
    from swifttransformer_amd.sampling import SamplingParams
    folder, cfg, w = models["A"]
    prompts = [tiny.prompt(n, cfg["vocab"], 70 + i) for i, n in enumerate((30, 26, 21, 5))]
    sp = SamplingParams(max_new_tokens=20, ignore_eos=True)
    tight = Engine(folder, dtype="fp32", page_size=4, num_pages=19, max_seqs=2, max_batched_tokens=64, prefill_chunk=9)
    outs = tight.generate(prompts, sp)
    assert tight.stats.preemptions >= 1, "the pool was meant to run out"
    for p, o in zip(prompts, outs):
        assert o == plain.generate(cfg, w, p, 20), f"prompt of {len(p)} tokens"
    tight.runner.manager.check_invariants()
    assert tight.runner.manager.num_free_slots == 2


def test_trace_replay_command_line_and_a_named_size(models, tmp_path):
    import subprocess
    import sys
    folder, cfg, w = models["B"]
    seqs = {"x": tiny.prompt(21, cfg["vocab"], 60), "y": tiny.prompt(9, cfg["vocab"], 61)}
    refs = {r: plain.logits(cfg, w, s).numpy() for r, s in seqs.items()}
    steps = [{"step": 0, "entries": [{"id": "x", "tokens": seqs["x"][:13], "want": [0, 12]}], "end": []},
             {"step": 1, "entries": [{"id": "y", "tokens": seqs["y"][:8], "want": []},
                                     {"id": "x", "tokens": seqs["x"][13:15], "want": [1]}], "end": []},
             {"step": 2, "entries": [{"id": "x", "tokens": seqs["x"][15:], "want": [5]},
                                     {"id": "y", "tokens": seqs["y"][8:], "want": [0]}], "end": ["x", "y"]}]
    out = str(tmp_path / "out")
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    r = subprocess.run([sys.executable, os.path.join(root, "bin", "trace_run"), "--model", folder, "--dtype", "float32",
                        "--out", out, "--max-tokens", "64", "--page-size", "2"],
                       input="\n".join(json.dumps(s) for s in steps) + "\n", capture_output=True, text=True, timeout=300)
    assert r.returncode == 0, r.stderr[-2000:]
    assert [l for l in r.stdout.split("\n") if l.startswith("done")] == ["done 0", "done 1", "done 2"]
    V = cfg["vocab"]
    got = {n: np.fromfile(os.path.join(out, f"{n}.f32"), dtype="<f4").reshape(-1, V) for n in (0, 1, 2)}
    check(torch.from_numpy(got[0]), refs["x"][[0, 12]], torch.float32, "step 0")
    check(torch.from_numpy(got[1]), refs["x"][[14]], torch.float32, "step 1")
    check(torch.from_numpy(got[2]), np.stack([refs["x"][20], refs["y"][8]]), torch.float32, "step 2")
    inp = tmp_path / "prompts.txt"
    inp.write_text(" ".join(map(str, seqs["y"])) + "\n")
    r = subprocess.run([sys.executable, os.path.join(root, "bin", "run_opt"), folder, "auto", "fp32", str(inp),
                        "--max-new-tokens", "5", "--ignore-eos", "--block-size", "2", "--num-blocks", "64", "--max-seqs", "2"],
                       capture_output=True, text=True, timeout=300)
    assert r.returncode == 0, r.stderr[-2000:]
    want = plain.generate(cfg, w, seqs["y"], 5)
    assert ")" + "".join(f"{t} " for t in want) in r.stdout
    # a named size with random weights, from its folder: the same logits as the plain model
    from swifttransformer_amd.config.registry import hyper_param_by_name
    from swifttransformer_amd.weights import write_random_model
    hp = hyper_param_by_name("fefozen_125m", num_layers=4, vocab=211, max_positions=128)
    d = write_random_model(hp, str(tmp_path / "named"), seed=3)
    cfg3, w3 = plain.load_folder(d)
    seq = tiny.prompt(40, 211, 8)
    runner = make_runner(d, "float32", 16, 8)
    run_schedule(runner, {0: seq}, {0: plain.logits(cfg3, w3, seq).numpy()}, [[(0, 33)]] + [[(0, 1)]] * 7, "float32", "named size",
                 loosen=3.0)
