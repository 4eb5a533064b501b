"""Fiterax on the GPU against the plain implementation: each new or extended kernel alone, then the engine on small
models in float32 and bfloat16: every layer, whole prompts, decoding through state and cache, portions down to two tokens,
unequal batches with slots and pages used again, first tokens, keys far back and at page borders, portions at the edges
of the memory's chunks, long decoding, greedy generation through ``Engine``, the replay loop and a named size."""
import copy
import json
import os

import numpy as np
import pytest
import torch

import plain_fiterax as plain
import tiny_fiterax as tiny
from test_pupalix_gpu import _paged
from test_zimorax_gpu import DEV, DTYPES, F64, check, dev, items_ctx, make_runner, rounded, run_schedule

pytestmark = pytest.mark.gpu


def _with_padding(ctx):
    """The same batch with one padding row behind it."""
    ti, il, off, sl = ctx
    return torch.cat([ti, torch.tensor([-1], dtype=torch.int32, device=DEV)]), il, off, sl


# ------------------------------------------------------------------ kernels alone
@pytest.mark.parametrize("dtype", list(DTYPES))
@pytest.mark.parametrize("W,groups", [(64, 4), (90, 3), (2048, 4), (48, 48), (130, 1), (2052, 3)])
def test_norm_in_groups_of_all_and_of_picked_rows(dtype, W, groups):
    from swifttransformer_amd.ops import kernels as K
    g = torch.Generator().manual_seed(W + groups)
    dt = DTYPES[dtype]
    x = torch.randn(9, W, generator=g, dtype=F64) * torch.linspace(0.01, 5.0, W, dtype=F64)
    gain = 1.0 + 0.3 * torch.randn(W, generator=g, dtype=F64)
    want = plain.group_rms(x, gain, groups, 1e-4).numpy()
    t, f = torch.empty((9, W), dtype=dt, device=DEV), torch.empty((9, W), device=DEV)
    K.group_rms(dev(x), dev(gain), groups, 1e-4, out_t=t, out_f32=f)
    check(t, want, dt, "storage type")
    check(f, want, torch.float32, "float")
    rows = torch.tensor([8, -1, 0, 3, 3], dtype=torch.int32, device=DEV)
    out = torch.empty((5, W), device=DEV)
    K.group_rms(dev(x), dev(gain), groups, 1e-4, rows=rows, out_f32=out)
    picked = want[[8, 0, 0, 3, 3]].copy()
    picked[1] = 0.0
    check(out, picked, torch.float32, "picked rows")


@pytest.mark.parametrize("dtype", list(DTYPES))
@pytest.mark.parametrize("W,groups,taps,sides", [(64, 4, 3, 2), (90, 3, 5, 2), (2048, 4, 3, 2), (130, 1, 1, 2), (96, 2, 8, 1),
                                                 (5000, 4, 2, 2), (72, 8, 4, 1), (300, 5, 8, 2)])
def test_norm_and_filter_in_portions_on_used_slots(dtype, W, groups, taps, sides):
    """Three requests in unequal portions over several steps: every row and the state each step leaves, beside a
    padding row and slots of others that stay as they are; an own filter and gain a side."""
    from swifttransformer_amd.ops import kernels as K
    g = torch.Generator().manual_seed(W * 10 + taps)
    dt, eps = DTYPES[dtype], 1e-5
    seqs = {s: torch.randn(n, W, generator=g, dtype=F64) * 3.0 for s, n in ((4, 23), (1, 9), (0, 5))}
    gains = [1.0 + 0.3 * torch.randn(W, generator=g, dtype=F64) for _ in range(sides)]
    filters = [0.5 * torch.randn(W, taps, generator=g, dtype=F64) for _ in range(sides)]
    normed = [{s: plain.group_rms(x, gains[i], groups, eps) for s, x in seqs.items()} for i in range(sides)]
    want = [{s: plain.input_conv(n, filters[i]) for s, n in normed[i].items()} for i in range(sides)]
    states = [torch.full((6, taps - 1, W), 7.5, device=DEV) for _ in range(sides)]
    for st in states:
        st[[4, 1, 0]] = 0.0                       # what admission leaves
    done = {s: 0 for s in seqs}
    for step in ([(4, 2), (1, 1)], [(1, 1), (4, 1), (0, 1)], [(4, 11), (1, 1)], [(0, 2), (1, 5), (4, 1)], [(4, 8), (0, 2), (1, 1)]):
        lens, slots = [n for _, n in step], [s for s, _ in step]
        x = torch.cat([seqs[s][done[s]:done[s] + n] for s, n in step] + [torch.full((1, W), float("nan"), dtype=F64)])
        single = all(n == 1 for n in lens)
        outs = K.group_norm_conv(dev(x), [(dev(gains[i]), dev(filters[i].t()), states[i] if taps > 1 else None) for i in range(sides)],
                                 groups, eps, _with_padding(items_ctx(lens, slots)), dt, all_single=single)
        for i in range(sides):
            ref = torch.cat([want[i][s][done[s]:done[s] + n] for s, n in step] + [torch.zeros(1, W, dtype=F64)])
            check(outs[i], ref.numpy(), dt, f"side {i} step {step}")
        for s, n in step:
            done[s] += n
            for i in range(sides):
                for b in range(1, taps):
                    p = done[s] - b
                    ref = normed[i][s][p] if p >= 0 else torch.zeros(W, dtype=F64)
                    check(states[i][s, taps - 1 - b][None], ref[None].numpy(), torch.float32, f"state {b} rows back of slot {s}")
    for st in states:
        assert (st[[2, 3, 5]] == 7.5).all()


@pytest.mark.parametrize("dtype", list(DTYPES))
def test_norm_and_filter_at_prompt_sizes(dtype):
    """Enough rows that a workgroup takes several, items starting in the middle of one."""
    from swifttransformer_amd.ops import kernels as K
    g = torch.Generator().manual_seed(5)
    dt, W, groups, taps = DTYPES[dtype], 64, 4, 4
    lens, slots = [1, 2, 1301, 1, 3, 770], [3, 0, 5, 1, 2, 4]
    xs = [torch.randn(n, W, generator=g, dtype=F64) for n in lens]
    gain, flt = 1.0 + 0.3 * torch.randn(W, generator=g, dtype=F64), 0.5 * torch.randn(W, taps, generator=g, dtype=F64)
    before = [torch.randn(taps - 1, W, generator=g, dtype=F64) for _ in lens]      # the normed rows of earlier steps
    state = torch.zeros((6, taps - 1, W), device=DEV)
    for b, s in zip(before, slots):
        state[s] = dev(b)
    out = K.group_norm_conv(dev(torch.cat(xs)), [(dev(gain), dev(flt.t()), state)], groups, 1e-5, items_ctx(lens, slots), dt)[0]
    refs = []
    for x, b in zip(xs, before):
        n = plain.group_rms(x, gain, groups, 1e-5)
        refs.append(plain.input_conv(torch.cat([b, n]), flt)[taps - 1:])
    check(out, torch.cat(refs).numpy(), dt, "rows")
    for x, b, s in zip(xs, before, slots):
        check(state[s], torch.cat([b, plain.group_rms(x, gain, groups, 1e-5)])[-(taps - 1):].numpy(), torch.float32, f"slot {s}")


@pytest.mark.parametrize("dtype", list(DTYPES))
@pytest.mark.parametrize("H,G,d,vd,rot,cap,gated,ps", [(4, 2, 16, 24, 8, 5.0, True, 4), (3, 3, 10, 6, 10, 0.0, True, 2),
                                                       (8, 1, 32, 32, 0, 30.0, False, 16), (2, 1, 100, 64, 40, 3.0, True, 16),
                                                       (6, 2, 48, 80, 2, 20.0, True, 8), (5, 1, 24, 250, 24, 9.0, True, 4)])
def test_turned_unit_queries_and_keys_into_pages_and_capped_gated_attention(dtype, H, G, d, vd, rot, cap, gated, ps):
    """Turn, norm, factor and page write (in two portions, entries padded), then every row's attention through the row
    kernel with and without key splits and through the tile kernel, against the plain equations of the same inputs."""
    from swifttransformer_amd.engine.batch import StepItem
    from swifttransformer_amd.ops import kernels as K
    from swifttransformer_amd.parts.attention import plan_tiles
    from swifttransformer_amd.parts.position import rotary_frequencies
    g = torch.Generator().manual_seed(H * 100 + d)
    dt = DTYPES[dtype]
    lens, eps, scale, base = [150, 3, 67], 1e-5, 1.5 / d ** 0.5, 40.0
    pad = -(-max(d, vd) // 16) * 16
    bt, num_pages = _paged(lens, ps, g)
    k_cache = torch.full((num_pages, G, ps, pad), float("nan"), dtype=dt, device=DEV)
    v_cache = torch.full((num_pages, G, ps, pad), float("nan"), dtype=dt, device=DEV)
    factor = 1.0 + 0.4 * torch.randn(H, generator=g)
    freq = dev(torch.tensor(rotary_frequencies(rot, base)[0])) if rot else None
    width = (H + G) * d + G * vd
    qs, gates, refs = [], [], []
    for b, n in enumerate(lens):
        proj = torch.randn(n, width + H + 3, generator=g) * 2.0              # wider than q, k and v: a slice of a product
        q64, k64 = proj[:, :H * d].to(F64).view(n, H, d), proj[:, H * d:(H + G) * d].to(F64).view(n, G, d)
        v64 = proj[:, (H + G) * d:width].to(F64).view(n, G, vd)
        part = []
        for a, e in ((0, n // 2), (n // 2, n)):                               # two portions
            if e > a:
                item = torch.full((e - a,), b, dtype=torch.int32, device=DEV)
                pos = torch.arange(a, e, dtype=torch.int32, device=DEV)
                part.append(K.unit_qk_write(dev(proj)[a:e], H, G, d, vd, eps, freq, dev(factor), k_cache, v_cache, item, pos,
                                            bt.to(DEV)))
        q_dev = torch.cat(part)
        turn = (lambda x: plain.turn_halves(x, rot, base)) if rot else (lambda x: x)
        qn = plain.rms(turn(q64), eps) * factor.to(F64)[:, None]
        kn = plain.rms(turn(k64), eps)
        check(q_dev.view(n, H, pad)[:, :, :d].reshape(n, H * d), qn.reshape(n, H * d).numpy(), dt, f"queries of request {b}", loosen=2.0)
        assert float(q_dev.view(n, H, pad)[:, :, d:].abs().sum()) == 0.0
        at = [(int(bt[b, p // ps]), p % ps) for p in range(n)]
        got_k = torch.stack([k_cache[page, :, r] for page, r in at])
        got_v = torch.stack([v_cache[page, :, r] for page, r in at])
        check(got_k[:, :, :d].reshape(n, -1), kn.reshape(n, -1).numpy(), dt, f"keys of request {b}", loosen=2.0)
        check(got_v[:, :, :vd].reshape(n, -1), v64.reshape(n, -1).numpy(), dt, f"values of request {b}")
        assert float(got_k[:, :, d:].abs().sum()) == 0.0 and float(got_v[:, :, vd:].abs().sum()) == 0.0
        # the plain attention on what was stored
        qq = q_dev.view(n, H, pad)[:, :, :d].cpu().to(F64)
        kk = got_k[:, :, :d].cpu().to(F64).repeat_interleave(H // G, dim=1)
        vv = got_v[:, :, :vd].cpu().to(F64).repeat_interleave(H // G, dim=1)
        s = torch.matmul(qq.transpose(0, 1), kk.permute(1, 2, 0)) * scale
        s = cap * torch.tanh(s / cap) if cap else s
        i, j = torch.arange(n)[:, None], torch.arange(n)[None, :]
        o = torch.matmul(torch.softmax(s.masked_fill((j > i)[None], float("-inf")), -1), vv.transpose(0, 1)).transpose(0, 1)
        z = proj[:, width:width + H]
        refs.append(o * torch.sigmoid(z.to(F64))[:, :, None] if gated else o)
        gates.append(proj[:, width - 1:width + H + 1])
        qs.append(q_dev)
    q_all, ref = torch.cat(qs), torch.cat(refs).reshape(-1, H * vd).numpy()
    gate = dev(torch.cat(gates))[:, 1:1 + H] if gated else None               # rows of any stride
    ti = torch.tensor([b for b, n in enumerate(lens) for _ in range(n)], dtype=torch.int32, device=DEV)
    pos = torch.tensor([p for n in lens for p in range(n)], dtype=torch.int32, device=DEV)
    cut = lambda out: out.view(-1, H, pad)[:, :, :vd].reshape(-1, H * vd)
    for splits in (1, 3):
        got = K.attention_rows(q_all, k_cache, v_cache, ti, pos, bt.to(DEV), H, scale, num_splits=splits, softcap=cap, head_gate=gate)
        check(cut(got), ref, dt, f"rows, {splits} splits", loosen=2.0)
        ids = torch.tensor([151, 5, -1, 219], dtype=torch.int32, device=DEV)
        out = torch.full_like(got, 3.0)
        K.attention_rows(q_all, k_cache, v_cache, ti, pos, bt.to(DEV), H, scale, num_splits=splits, softcap=cap, head_gate=gate,
                         row_ids=ids, out=out)
        check(cut(out)[[151, 5, 219]], ref[[151, 5, 219]], dt, "picked rows", loosen=2.0)
        assert (out[[0, 1, 150]] == 3.0).all()
    plan = plan_tiles([StepItem(slot=b, start=0, tokens=[0] * n) for b, n in enumerate(lens)], 8)
    mk = lambda a: torch.tensor(np.asarray(a), dtype=torch.int32, device=DEV)
    out = torch.zeros_like(q_all)
    K.attention_prefill(q_all, k_cache, v_cache, mk(plan.arrays["tile_item"]), mk(plan.arrays["tile_q0"]),
                        mk(np.concatenate([[0], np.cumsum(lens)[:-1]])), mk([0] * len(lens)), mk(lens), bt.to(DEV), H, scale, out=out,
                        softcap=cap, head_gate=gate)
    rows = [t for t, b in enumerate(ti.tolist()) if lens[b] >= 8]
    check(cut(out)[rows], ref[rows], dt, "tiles", loosen=2.0)


def _memory_case(H, dk, dv, n, g, cap, dtype, spread=1.0):
    """A request's projected rows and what the plain memory makes of them (bfloat16 leaves the rows' floats alone)."""
    q, v, gate = (torch.randn(n, H, w, generator=g) for w in (dk, dv, dv))
    k = 0.7 * q + 0.5 * torch.randn(n, H, dk, generator=g)
    zi, zf = spread * 3.0 * torch.randn(n, H, generator=g), spread * (2.0 + 4.0 * torch.randn(n, H, generator=g))
    rows = torch.cat([t.reshape(n, -1) for t in (q, k, v, gate, zi, zf)], dim=1)
    return rows, (q, k, v, gate, zi, zf)


def _memory_ref(parts, bi, bf, gain, cap, eps):
    q, k, v, gate, zi, zf = (t.to(F64) for t in parts)
    n, H, dk = q.shape
    i = cap * torch.tanh((zi + bi.to(F64)) / cap)
    f = torch.nn.functional.logsigmoid(cap * torch.tanh((zf + bf.to(F64)) / cap))
    o = plain.rms(plain.mlstm_memory(q * dk ** -0.5, k, v, i, f), eps)
    return o.reshape(n, -1) * gain.to(F64) * torch.sigmoid(gate).reshape(n, -1)


@pytest.mark.parametrize("dtype", list(DTYPES))
@pytest.mark.parametrize("H,dk,dv,cap", [(2, 12, 20, 9.0), (3, 5, 7, 15.0), (4, 72, 40, 2.0), (1, 16, 64, 12.0), (2, 64, 128, 15.0),
                                         (1, 130, 200, 6.0), (2, 256, 256, 15.0), (1, 33, 65, 10.0), (5, 1, 1, 4.0)])
def test_matrix_memory_whole_by_tokens_and_in_portions(dtype, H, dk, dv, cap):
    """One request whole, token by token, in portions at and off the chunks' borders and mixed, each from a cleared
    slot among others that must not move; then two unequal requests side by side."""
    from swifttransformer_amd.ops import kernels as K
    g = torch.Generator().manual_seed(H * 1000 + dk)
    dt, eps, n = DTYPES[dtype], 1e-5, 150
    bi, bf = torch.randn(H, generator=g), torch.randn(H, generator=g)
    gain = 1.0 + 0.2 * torch.randn(H * dv, generator=g)
    rows, parts = _memory_case(H, dk, dv, n, g, cap, dtype)
    ref = _memory_ref(parts, bi, bf, gain, cap, eps).numpy()
    slot_floats = K.memory_slot(H, dk, dv)
    wide = torch.cat([rows, torch.full((n, 5), float("nan"))], dim=1)          # rows of a product filled up behind
    args = (dev(bi), dev(bf), dev(gain))

    def run(proj, lens, slots, state, single=False):
        return K.matrix_memory(proj, *args, state, items_ctx(lens, slots), H, dk, dv, cap, eps, dt, all_single=single)
    finals = []
    for cuts in ([n], [1] * n, [64, 64, 22], [63, 1, 2, 65, 1, 18], [2] * 40 + [1] * 6 + [64]):
        state = torch.full((4, slot_floats), 5.0, device=DEV)
        state[2] = 0.0
        at, outs = 0, []
        for c in cuts:
            outs.append(run(dev(wide)[at:at + c], [c], [2], state, single=c == 1 and at % 3 != 1))   # (a chunk of one row too)
            at += c
        check(torch.cat(outs), ref, dt, f"cuts {cuts[:6]}", loosen=3.0)
        assert (state[[0, 1, 3]] == 5.0).all()
        finals.append(state[2].clone())
    used = H * (dk * dv + dk + 1)
    for f in finals[1:]:
        check(f[None, :used], finals[0][None, :used].cpu().numpy(), torch.float32, "final state", loosen=3.0)
    # two requests of unequal portions, an item without rows between them, a slot used before
    rows2, parts2 = _memory_case(H, dk, dv, 71, g, cap, dtype)
    ref2 = _memory_ref(parts2, bi, bf, gain, cap, eps).numpy()
    state = torch.zeros((3, slot_floats), device=DEV)
    a = run(torch.cat([dev(rows)[:100], dev(rows2)[:1]]), [100, 0, 1], [1, -1, 0], state)
    b = run(torch.cat([dev(rows2)[1:70], dev(rows)[100:]]), [69, 50], [0, 1], state)
    c = run(dev(rows2)[70:], [1], [0], state, single=True)
    check(torch.cat([a[:100], b[69:]]), ref, dt, "first of two", loosen=3.0)
    check(torch.cat([a[100:], b[:69], c]), ref2, dt, "second of two", loosen=3.0)


@pytest.mark.parametrize("zi,zf", [(20.0, -20.0), (-20.0, -20.0), (-20.0, 20.0), (20.0, 20.0), (0.0, 40.0)])
def test_matrix_memory_at_the_gates_ends(zi, zf):
    """Gates at their caps: a memory that forgets everything at once, one that keeps all of it, inputs that weigh next to
    nothing (the denominator's lower bound), in chunks and token by token."""
    from swifttransformer_amd.ops import kernels as K
    g = torch.Generator().manual_seed(3)
    H, dk, dv, n, cap, eps = 2, 16, 24, 140, 12.0, 1e-5
    rows, parts = _memory_case(H, dk, dv, n, g, cap, "float32", spread=0.2)
    parts = parts[:4] + (parts[4] + zi, parts[5] + zf)
    rows = torch.cat([t.reshape(n, -1) for t in parts], dim=1)
    zero, gain = torch.zeros(H), torch.ones(H * dv)
    ref = _memory_ref(parts, zero, zero, gain, cap, eps).numpy()
    for cuts in ([n], [70, 1, 69], [1] * n):
        state = torch.zeros((1, K.memory_slot(H, dk, dv)), device=DEV)
        at, outs = 0, []
        for c in cuts:
            outs.append(K.matrix_memory(dev(rows)[at:at + c], dev(zero), dev(zero), dev(gain), state, items_ctx([c], [0]), H, dk, dv,
                                        cap, eps, torch.float32, all_single=c == 1))
            at += c
        check(torch.cat(outs), ref, torch.float32, f"{cuts[:3]}", loosen=4.0)


@pytest.mark.parametrize("dtype", list(DTYPES))
@pytest.mark.parametrize("E,top,W,F,T", [(6, 2, 64, 24, 37), (5, 5, 90, 20, 9), (8, 1, 128, 40, 300), (4, 3, 48, 16, 150),
                                         (8, 2, 256, 192, 420), (80, 4, 64, 16, 21), (12, 4, 72, 136, 330)])
def test_experts_without_a_gate_chosen_by_corrected_and_weighted_by_normalised_sigmoids(dtype, E, top, W, F, T):
    from swifttransformer_amd.ops import kernels as K
    g = torch.Generator().manual_seed(E * 10 + top)
    dt, scale = DTYPES[dtype], 1.7
    x = rounded(torch.randn(T, W, generator=g), dtype)
    up, down = rounded(torch.randn(E, F, W, generator=g) * 1.5 / W ** 0.5, dtype), rounded(torch.randn(E, W, F, generator=g) / F ** 0.5, dtype)
    # scores a permutation of well separated levels a row (no close call), some moved by corrections of another order
    levels = torch.linspace(0.1, 0.9, E, dtype=F64)
    s = torch.stack([levels[torch.randperm(E, generator=g)] for _ in range(T)])
    correction = torch.zeros(E)
    correction[E // 2], correction[0] = 1.0, -1.0
    logits = torch.log(s / (1 - s)).to(torch.float32)
    ref = torch.zeros(T, W, dtype=F64)
    for t in range(T):
        for e, wgt in plain.route(logits[t].to(F64), correction.to(F64), top, scale):
            ref[t] += wgt * (plain.gelu(x[t] @ up[e].T) @ down[e].T)
    item = torch.zeros(T, dtype=torch.int32)
    item[T // 2] = -1                                           # a padding row
    kw = dict(top=top, token_item=item.to(DEV), style="sigmoid_output", correction=dev(correction), scale=scale)
    ref[T // 2] = 0.0
    got = K.routed_experts(dev(x, dt), dev(logits), None, dev(up, dt), dev(down, dt), None, **kw)
    check(got, ref.numpy(), dt, "the sum alone", loosen=2.0)
    base = torch.randn(T, W, generator=g)
    got = K.routed_experts(dev(x, dt), dev(logits), None, dev(up, dt), dev(down, dt), dev(base), out_scale=0.6, **kw)
    check(got, (0.6 * ref + base.to(F64)).numpy(), dt, "onto a stream", loosen=2.0)


@pytest.mark.parametrize("dtype", list(DTYPES))
@pytest.mark.parametrize("M,N,K_", [(1, 64, 128), (8, 2048, 512), (16, 96, 90), (40, 256, 192), (200, 192, 320), (7, 50, 33)])
def test_a_bias_behind_the_factor_on_every_product_path(dtype, M, N, K_):
    from swifttransformer_amd.ops import kernels as K
    g = torch.Generator().manual_seed(M + N)
    dt = DTYPES[dtype]
    x, w = rounded(torch.randn(M, K_, generator=g), dtype), rounded(torch.randn(N, K_, generator=g) / K_ ** 0.5, dtype)
    b, r = torch.randn(N, generator=g), torch.randn(M, N, generator=g)
    want = (r.to(F64) + 0.3 * (x @ w.T) + b.to(F64)).numpy()
    for algo in (0, 1):
        got = K.gemm(dev(x, dt), dev(w, dt), bias=dev(b), residual=dev(r), out_f32=True, out_scale=0.3, bias_unscaled=True, algo=algo)
        check(got, want, torch.float32 if dtype == "float32" else dt, f"algo {algo}")
    got = K.gemm(dev(x, dt), dev(w, dt), bias=dev(b), residual=dev(r), out_f32=True, out_scale=0.3)
    check(got, (r.to(F64) + 0.3 * (x @ w.T + b.to(F64))).numpy(), dt, "bias inside the factor")


# ------------------------------------------------------------------ the engine on small models
@pytest.fixture(scope="module")
def models(tmp_path_factory):
    root = tmp_path_factory.mktemp("fiterax")
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
            seen.append(_orig(x32, *a, **kw).clone())
            return seen[-1]
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
def test_portions_at_the_edges_of_the_memorys_chunks_beside_others(models, dtype):
    folder, cfg, w = models["A"]
    seqs = {0: tiny.prompt(330, cfg["vocab"], 7), 1: tiny.prompt(40, cfg["vocab"], 8)}
    refs = {r: plain.logits(cfg, w, s).numpy() for r, s in seqs.items()}
    ps = tiny.PAGE_SIZE["A"]
    runner = make_runner(folder, dtype, ps, -(-330 // ps) + -(-40 // ps) + 2, record_after=2)
    schedule = [[(0, 63), (1, 20)], [(1, 1), (0, 65)], [(0, 1), (1, 1)], [(1, 2), (0, 64)], [(0, 16), (1, 16)]] + \
               [[(0, 1)]] * 50 + [[(0, 2)], [(0, 69)]]
    run_schedule(runner, seqs, refs, schedule, dtype, f"A {dtype} mixed", loosen=2.0)


def _single_layer(cfg0, w0, index, tmp_path, change):
    """A model made of layer ``index`` of ``cfg0`` alone (as its layer 0), without feed-forward."""
    cfg = copy.deepcopy(cfg0)
    cfg["layers"] = [dict(cfg["layers"][index], mlp=None)]
    pre = f"l{index}."
    w = {("l0." + k[len(pre):] if k.startswith(pre) else k): v.to(torch.float32).clone() for k, v in w0.items()
         if (k.startswith(pre) and ".mlp." not in k and "norm2" not in k and "canon2" not in k) or k in ("embed", "head", "final.norm")}
    change(cfg["layers"][0]["mixer"], w)
    folder = tiny.write_folder(cfg, str(tmp_path / "peaked"), 0, weights=w)
    return (folder,) + plain.load_folder(folder)


@pytest.mark.parametrize("dtype", list(DTYPES))
@pytest.mark.parametrize("name,index,ps", [("A", 0, 4), ("A", 2, 16), ("C", 0, 8)])
def test_peaked_attention_far_back_and_at_page_borders(models, tmp_path, dtype, name, index, ps):
    """An attention alone, its scores scaled up (and its cap raised) so that the softmax picks single keys: a key that is
    wrongly seen or missed, or turned by a wrong position, moves the row.  The plain model's own parts say which key each
    query weighs most: some far back, some at page borders, some the sequence's first."""
    _, cfg0, w0 = models[name]
    boost = 30.0 if dtype == "float32" else 3.0

    def change(m, w):
        m["scale"] = m["scale"] * boost
        if m.get("softcap"):
            m["softcap"] = 40.0 * boost
    folder, cfg, w = _single_layer(cfg0, w0, index, tmp_path, change)
    T = 330
    seq = tiny.prompt(T, cfg["vocab"], 5)
    ref = plain.logits(cfg, w, seq).numpy()
    m, eps = cfg["layers"][0]["mixer"], cfg["norm"]["eps"]
    H, G, d = m["heads"], m["kv_heads"], m["dim"]
    x = w["embed"][torch.tensor(seq)] * cfg["embedding"]["scale"]
    h = plain.input_conv(plain.group_rms(x, w["l0.norm1"], cfg["norm"]["groups"], eps), w["l0.canon1"])
    q, k = (h @ w["l0.mix.q"].T + w["l0.mix.q.b"]).view(T, H, d), (h @ w["l0.mix.k"].T + w["l0.mix.k.b"]).view(T, G, d)
    if m.get("rot"):
        q, k = (plain.turn_halves(t, m["rot"]["dims"], m["rot"]["base"]) for t in (q, k))
    q, k = plain.rms(q, eps), plain.rms(k, eps)
    i, j = torch.arange(T)[:, None], torch.arange(T)[None, :]
    best = []
    for n in range(H):
        s = ((q[:, n] @ k[:, n // (H // G)].T) * w["l0.mix.temp"][n]).masked_fill(j > i, float("-inf"))
        best += [(t, int(s[t].argmax())) for t in range(T)]
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
def test_a_memory_that_keeps_a_token_for_long(models, tmp_path, dtype):
    """A memory alone that forgets next to nothing, so that the first tokens still show hundreds of tokens later; a
    state that was lost, cut or mixed with another request's moves every later row."""
    _, cfg0, w0 = models["A"]

    def change(m, w):
        w["l0.mix.f"] *= 0.0
        w["l0.mix.f.b"] = torch.full_like(w["l0.mix.f.b"], 8.0)
        w["l0.mix.i"] *= 3.0                               # a few tokens outweigh the rest
        w["l0.mix.o"] *= 4.0
    folder, cfg, w = _single_layer(cfg0, w0, 1, tmp_path, change)
    seqs = {0: tiny.prompt(300, cfg["vocab"], 5), 1: tiny.prompt(120, cfg["vocab"], 6)}
    refs = {r: plain.logits(cfg, w, s).numpy() for r, s in seqs.items()}
    other = plain.logits(cfg, w, seqs[1][:60] + seqs[0][60:]).numpy()
    assert np.abs(other[299] - refs[0][299]).max() > 0.3 * refs[0][299].std()       # the first tokens show at the end
    runner = make_runner(folder, dtype, 4, 120, record_after=2, max_seqs=2)
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
    computed again later in a slot that held another request's memory and filter inputs."""
    from swifttransformer_amd.engine.engine import Engine
    from swifttransformer_amd.sampling import SamplingParams
    folder, cfg, w = models["A"]
    prompts = [tiny.prompt(n, cfg["vocab"], 70 + i) for i, n in enumerate((30, 26, 21, 5))]
    sp = SamplingParams(max_new_tokens=20, ignore_eos=True)
    # (two paged groups: the attentions' entries differ)
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
    hp = hyper_param_by_name("fiterax_125m", num_layers=3, vocab=211, max_positions=128)
    d = write_random_model(hp, str(tmp_path / "named"), seed=3)
    cfg3, w3 = plain.load_folder(d)
    seq = tiny.prompt(40, 211, 8)
    runner = make_runner(d, "float32", 16, 8)
    run_schedule(runner, {0: seq}, {0: plain.logits(cfg3, w3, seq).numpy()}, [[(0, 33)]] + [[(0, 1)]] * 7, "float32", "named size",
                 loosen=3.0)
