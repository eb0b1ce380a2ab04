"""Semezen on the GPU against the plain implementation (``plain_semezen``): each mechanism's kernels alone, with inputs made so
that a fault shows (one key that stands out just inside and just outside a window, a write that must be recalled after hundreds
of tokens, a row of streams that only one entry of the mix reaches), then whole models under every cutting, batching, page and
slot reuse, long decoding, and greedy generation through the engine's own entry point."""
import json
import os
from types import SimpleNamespace

import numpy as np
import pytest
import torch

import plain_semezen as P
import tiny_semezen as TS
from gpu_tools import (DEV, PagedKV, RouteRecorder, attention_ctx, close, cut_steps, dev32, in_steps, live_token_need, make_part, paged, randn,
                       run_paged_part, run_trace, state_ctx)
from tiny_models import random_tokens

pytestmark = pytest.mark.gpu
DTYPES = ["float32", "bfloat16"]
TORCH = {"float32": torch.float32, "bfloat16": torch.bfloat16}
F64 = torch.float64


def act_tol(dtype):
    return 3e-5 if dtype == "float32" else 1.2e-2


# ----------------------------------------------------------------------------- streams side by side
def streams_case(T, n, D, seed=1):
    X = randn(T, n, D, seed=seed, scale=2.0)
    y, mix, out = randn(T, D, seed=seed + 1), randn(n, n, seed=seed + 2) * 0.4 + torch.eye(n, dtype=F64), randn(n, seed=seed + 3)
    read, w = randn(n, seed=seed + 4), randn(D, seed=seed + 5) * 0.3 + 1.0
    new = torch.stack(P.mix_streams([X[:, s] for s in range(n)], y, mix, out), dim=1)
    post = torch.cat([out, mix.reshape(-1)])
    h = lambda Z, eps: P.rms_norm((read[:, None] * Z).sum(1), w, eps)
    return X, y, post, read, w, new, h


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("T,n,D", [(7, 1, 64), (5, 2, 90), (9, 3, 520), (600, 4, 256), (4, 4, 2048), (6, 5, 100), (3, 9, 72), (2, 16, 64), (5, 4, 3072),
                                   (3, 3, 4100), (2, 2, 16384), (3, 12, 6000)])
def test_update_and_next_norm_of_streams(dtype, T, n, D):
    from photon_infer_amd import ops
    eps = 1e-3
    X, y, post, read, w, new, h = streams_case(T, n, D)
    rows = torch.tensor([T - 1, 0, T // 2], dtype=torch.int32, device=DEV)
    kw = dict(h_dtype=TORCH[dtype], read=dev32(read), norm=dev32(w), eps=eps)
    x = dev32(X)
    close(ops.hyper_streams(x, **kw), h(X, eps), "h alone", act_tol(dtype))
    close(x, X, "h alone leaves the streams", 1e-6)
    close(ops.hyper_streams(x, y=dev32(y), post=dev32(post), **kw), h(new, eps), "update, then h", act_tol(dtype))
    close(x, new, "updated streams")
    x = dev32(X)
    close(ops.hyper_streams(x, y=dev32(y), post=dev32(post), rows=rows, **kw), h(new, eps)[rows.cpu().long()], "update and h of chosen rows", act_tol(dtype))
    close(x, X, "chosen rows leave the streams", 1e-6)
    assert ops.hyper_streams(x, y=dev32(y), post=dev32(post)) is None
    close(x, new, "update alone")


@pytest.mark.parametrize("splits", [2, 3, 8, 11])
def test_update_of_streams_adds_the_pieces_of_a_result(splits):
    from photon_infer_amd import ops
    from photon_infer_amd.ops.workspace import KernelWorkspace, Partials, PendingUpdate
    T, n, D = 5, 4, 640
    X, _, post, read, w, _, h = streams_case(T, n, D)
    pieces = randn(splits, T, D, seed=9)
    mix = post[n:].view(n, n)
    new = torch.stack(P.mix_streams([X[:, s] for s in range(n)], pieces.sum(0), mix, post[:n]), dim=1)
    ws = KernelWorkspace(DEV)
    y = torch.full((T, D), float("nan"), device=DEV)                    # unwritten while its pieces wait
    ws.pending = PendingUpdate(y, Partials(dev32(pieces), splits, T, D), accumulate=False)
    x = dev32(X)
    got = ops.hyper_streams(x, y=y, post=dev32(post), h_dtype=torch.float32, read=dev32(read), norm=dev32(w), eps=1e-5, ws=ws)
    assert ws.pending is None and ws.counts["added_by_streams"] == 1
    close(x, new, "streams")
    close(got, h(new, 1e-5), "h")
    ws.pending = PendingUpdate(y, Partials(dev32(pieces), splits, T, D), accumulate=False)
    ops.materialize(y, ws)                                              # somebody else needs the result itself
    close(y, pieces.sum(0), "written out")
    assert ws.pending is None


def test_every_stream_reaches_every_other_through_its_own_entry():
    """One entry of the mix at a time: from s to t, nothing else."""
    from photon_infer_amd import ops
    n, D = 3, 64
    X = randn(2, n, D, seed=1)
    for s in range(n):
        for t in range(n):
            mix = torch.zeros(n, n, dtype=F64)
            mix[s, t] = 2.0
            x = dev32(X)
            ops.hyper_streams(x, y=torch.zeros((2, D), device=DEV), post=dev32(torch.cat([torch.zeros(n, dtype=F64), mix.reshape(-1)])))
            want = torch.zeros_like(X)
            want[:, t] = 2.0 * X[:, s]
            close(x, want, f"from {s} to {t}", 1e-6)


def test_token_embedding_in_several_streams():
    from photon_infer_amd.parts import TokenEmbedding
    part = TokenEmbedding(11, 24, tensor_name="e", copies=3)
    table = randn(11, 24, seed=1).to(torch.bfloat16)
    part.load({"e": table.to(DEV)}, torch.bfloat16, torch.device(DEV))
    x = part.forward(torch.tensor([4, 0, 10], dtype=torch.int32, device=DEV))
    assert x.shape == (3, 3, 24) and all(torch.equal(x[:, s].cpu(), table.float()[[4, 0, 10]]) for s in range(3))


# ----------------------------------------------------------------------------- the token before
SHIFT_CUTS = ({"a": [40], "b": [9], "c": [1]}, {"a": [1], "b": [1], "c": [1]}, {"a": [2, 17, 1, 5], "b": [3, 2], "c": [1]}, {"a": [39, 1], "b": [1, 8], "c": [1]})


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("D", [64, 90, 1030])
def test_shift_towards_the_token_before_whole_and_cut(dtype, D):
    """Three requests in a step; state rows hold what the step before left; a step of single tokens goes through the streams'
    kernel, the others through the shift's own."""
    from photon_infer_amd import ops
    T, n, eps = {"a": 40, "b": 9, "c": 1}, 2, 1e-4
    share, w, read = torch.rand(D, generator=torch.Generator().manual_seed(5), dtype=F64), randn(D, seed=6) * 0.2 + 1, randn(n, seed=7)
    X = {k: randn(t, n, D, seed=10 + i) for i, (k, t) in enumerate(T.items())}
    plain_h = {k: P.rms_norm((read[:, None] * X[k]).sum(1), w, eps) for k in T}
    want = {k: P.shift_in(plain_h[k], share) for k in T}
    slot = {"a": 3, "b": 0, "c": 2}
    for cuts in SHIFT_CUTS:
        state = torch.zeros((4, D + 2), device=DEV)
        state[1] = 7.0                                                   # nobody's: stays
        got = {k: [] for k in T}
        for step in in_steps(T, cuts):
            lens = [j - i for _, i, j in step]
            ctx = state_ctx(lens, [slot[k] for k, _, _ in step])
            ctx.req_of_token = torch.repeat_interleave(torch.arange(len(lens), dtype=torch.int32), torch.tensor(lens)).int().to(DEV)
            ctx.all_decode = all(v == 1 for v in lens)
            x = dev32(torch.cat([X[k][i:j] for k, i, j in step]))
            kw = dict(read=dev32(read), norm=dev32(w), eps=eps)
            if ctx.all_decode:
                h = ops.hyper_streams(x, h_dtype=TORCH[dtype], shift=dev32(share), state=state[:, :D], ctx=ctx, **kw)
            else:
                h = ops.token_shift(ops.hyper_streams(x, h_dtype=torch.float32, **kw), dev32(share), state[:, :D], ctx, TORCH[dtype])
            for (k, _, _), part in zip(step, torch.split(h, lens)):
                got[k].append(part)
        for k in T:
            close(torch.cat(got[k]), want[k], f"{k} cut {cuts[k]}", act_tol(dtype))
            close(state[slot[k], :D], plain_h[k][-1], f"{k}: what is left for the next step", 1e-5)
        assert bool((state[1] == 7.0).all()) and bool((state[[0, 2, 3], D:] == 0).all())


# ----------------------------------------------------------------------------- minGRU
def gru_plain(proj, bias, W):
    z, u, g = proj[:, :W] + bias[:W], proj[:, W:2 * W] + bias[W:], proj[:, 2 * W:]
    return P.gru_walk(P.sigmoid(z), u) * P.silu(g)


def run_gru(T, data, bias, W, cuts, slot, dtype, splits=1):
    from photon_infer_amd import ops
    state = torch.zeros((4, W + 3), device=DEV)
    got = {k: [] for k in T}
    for step in in_steps(T, cuts):
        lens = [j - i for _, i, j in step]
        proj = torch.cat([data[k][i:j] for k, i, j in step])
        if splits > 1:          # as the pieces of a product split over k
            parts = randn(splits - 1, *proj.shape, seed=77)
            src = ops.Partials(dev32(torch.cat([parts, (proj - parts.sum(0))[None]])), splits, *proj.shape)
        else:
            src = dev32(proj)
        out = torch.empty((proj.shape[0], W), dtype=TORCH[dtype], device=DEV)
        ops.min_gru(out, src, dev32(bias), state_ctx(lens, [slot[k] for k, _, _ in step]), state[:, :W], W)
        for (k, _, _), part in zip(step, torch.split(out, lens)):
            got[k].append(part)
    assert bool((state[:, W:] == 0).all())
    return {k: torch.cat(v) for k, v in got.items()}, state


@pytest.mark.parametrize("W,splits", [(64, 1), (37, 1), (520, 3), (1100, 1)])
def test_min_gru_whole_in_portions_and_token_by_token(W, splits):
    T, slot = {"a": 83, "b": 10, "c": 33}, {"a": 3, "b": 1, "c": 0}
    data = {k: torch.cat([randn(t, W, seed=10 + i, scale=3.0) - 1.0, randn(t, 2 * W, seed=20 + i, scale=1.5)], dim=1) for i, (k, t) in enumerate(T.items())}
    bias = randn(2 * W, seed=1)
    want = {k: gru_plain(data[k], bias, W) for k in T}
    for cuts in ({"a": [83], "b": [10], "c": [33]}, {"a": [1], "b": [1], "c": [1]}, {"a": [2, 17, 1, 40], "b": [3, 2], "c": [32, 1]}, {"a": [9], "b": [10], "c": [2]}):
        for dtype in DTYPES:
            got, state = run_gru(T, data, bias, W, cuts, slot, dtype, splits)
            for k in T:
                close(got[k], want[k], f"{k} cut {cuts[k]} {dtype}", 3e-5 if dtype == "float32" else 1e-2)
            assert bool((state[2] == 0).all())


def test_min_gru_long_portions_beside_short_ones():
    W, T, slot = 96, {"a": 2500, "b": 700, "c": 9}, {"a": 0, "b": 2, "c": 3}
    data = {k: torch.cat([randn(t, W, seed=10 + i, scale=2.0) - 5.0, randn(t, 2 * W, seed=20 + i)], dim=1) for i, (k, t) in enumerate(T.items())}
    bias = randn(2 * W, seed=1)
    want = {k: gru_plain(data[k], bias, W) for k in T}
    for cuts in ({"a": [2500], "b": [700], "c": [9]}, {"a": [256, 1, 2100, 143], "b": [1, 699], "c": [1]}, {"a": [129, 31, 32, 33], "b": [44, 256], "c": [3]}):
        got, _ = run_gru(T, data, bias, W, cuts, slot, "float32")
        for k in T:
            close(got[k], want[k], f"{k} cut {cuts[k]}", 5e-5)


@pytest.mark.parametrize("decode", [False, True])
def test_min_gru_recalls_a_write_after_hundreds_of_tokens(decode):
    """Token 3 opens the gates and writes; then feature 0's gate is shut for good, feature 1's lets a thousandth in per token,
    feature 2's is as good as shut (e^-20): what is left after 900 tokens is known in closed form."""
    W, T = 4, 904
    z = torch.full((T, W), -200.0, dtype=F64)
    z[:, 1], z[:, 2] = float(np.log(1e-3 / (1 - 1e-3))), -20.0
    z[3] = 200.0
    u = torch.full((T, W), -200.0, dtype=F64)                 # candidates of zero ...
    u[3] = torch.tensor([4.0, 4.0, 4.0, -1.0], dtype=F64)     # ... but for token 3's
    g = torch.full((T, W), 30.0, dtype=F64)                   # silu(30) = 30
    out, _ = run_gru({"a": T}, {"a": torch.cat([z, u, g], dim=1)}, torch.zeros(2 * W, dtype=F64), W, {"a": [4, 300] + [1] * 600 if decode else [T]}, {"a": 1}, "float32")
    got = out["a"].double().cpu() / 30.0
    assert float(got[:3].abs().max()) < 1e-7
    left = T - 1 - 3
    close(got[3], torch.tensor([4.5, 4.5, 4.5, 1 / (1 + np.e)], dtype=F64), "the write itself", 1e-6)
    close(got[-1], torch.tensor([4.5, 4.5 * (1 - 1e-3) ** left, 4.5 * np.exp(-left * np.exp(-20.0)), 1 / (1 + np.e)], dtype=F64), "900 tokens later", 1e-5)


# ----------------------------------------------------------------------------- attention
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("sizes", [(4, 2, 16, 8, False), (4, 1, 64, 64, False), (6, 3, 12, 6, False), (3, 1, 10, 4, False), (2, 2, 80, 40, True), (1, 1, 96, 0, False),
                                   (2, 1, 256, 24, False), (2, 1, 320, 64, False), (4, 4, 32, 16, True)])
@pytest.mark.parametrize("T,splits", [(3, 1), (40, 1), (5, 4), (37, 3)])
def test_queries_keys_and_values_from_the_projection(dtype, sizes, T, splits):
    """Bias, rotation, norm per head, and the raw keys as values, into pages dealt out of order; gates as projected."""
    from photon_infer_amd import ops
    H, G, d, rd, inter = sizes
    page, eps, base, start, ng = 16, 1e-3, 50.0, 21, H * d
    tdt = TORCH[dtype]
    proj, bias = randn(T, (H + G) * d + ng, seed=1), randn((H + G) * d, seed=2)
    qk = (proj[:, :(H + G) * d] + bias).view(T, H + G, d)
    turned = qk.clone()
    for t in range(T):
        if rd and not inter:
            turned[t] = P.rotate_halves(qk[t], start + t, rd, base)
        elif rd:
            order = list(range(0, rd, 2)) + list(range(1, rd, 2)) + list(range(rd, d))          # neighbours as halves
            back = torch.empty_like(qk[t])
            back[:, order] = P.rotate_halves(qk[t][:, order], start + t, rd, base)
            turned[t] = back
    want = P.rms_norm(turned, None, eps)
    table, pages = paged([start + T], page, seed=3)
    kc, vc = torch.full((pages, G, page, d), 9.0, dtype=tdt, device=DEV), torch.full((pages, G, d, page), 9.0, dtype=tdt, device=DEV)
    ctx = attention_ctx([T], [start + T], tdt)
    rotary = (dev32(base ** (-2.0 * torch.arange(rd // 2, dtype=F64) / rd)), rd, inter) if rd else None
    if splits > 1:
        parts = randn(splits - 1, *proj.shape, seed=7)
        src = ops.Partials(dev32(torch.cat([parts, (proj - parts.sum(0))[None]])), splits, *proj.shape)
    else:
        src = dev32(proj)
    q = torch.empty((T, H * d), dtype=tdt, device=DEV)
    gates = ops.qk_rope_norm_write(q, src, dev32(bias), rotary, ctx, eps, H, G, d, ng, kc, vc, table, page)
    tol = 3e-5 if dtype == "float32" else 1e-2
    close(q, want[:, :H].reshape(T, -1), "queries", tol)
    close(gates, proj[:, (H + G) * d:], "gates", 2e-5)
    blk = [(int(table[0, (start + t) // page]), (start + t) % page) for t in range(T)]
    close(torch.stack([kc[p, :, s] for p, s in blk]), want[:, H:], "keys", tol)
    close(torch.stack([vc[p, :, :, s] for p, s in blk]), qk[:, H:], "values", tol)
    untouched = torch.ones((pages, page), dtype=torch.bool)
    for p, s in blk:
        untouched[p, s] = False
    assert bool((kc.cpu().transpose(1, 2)[untouched] == 9).all()) and bool((vc.cpu().permute(0, 3, 1, 2)[untouched] == 9).all())


def gated_reference(q, k, v, q_lens, kv_lens, scale, window, gate):
    """q [T, H, d] of several requests in a row, k / v per request [S, G, d], gate [T, H * d] as projected."""
    outs, row = [], 0
    for r, (n, kv) in enumerate(zip(q_lens, kv_lens)):
        H, G = q.shape[1], k[r].shape[1]
        o = torch.zeros(n, H, q.shape[2], dtype=F64)
        for h in range(H):
            g = h // (H // G)
            for i in range(n):
                p = kv - n + i
                lo = max(0, p - window + 1) if window else 0
                s = (k[r][lo:p + 1, g] @ q[row + i, h]) * scale
                w = torch.exp(s - s.max())
                o[i, h] = (w / w.sum()) @ v[r][lo:p + 1, g]
        outs.append(o.reshape(n, -1))
        row += n
    return torch.cat(outs) * P.sigmoid(gate)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("sizes,q_lens,kv_lens,window", [
    ((4, 2, 64), [70], [70], 0), ((4, 2, 64), [64], [2100], 0), ((4, 1, 128), [1, 1], [900, 33], 0), ((4, 1, 128), [1, 1], [900, 33], 40),
    ((8, 2, 32), [1, 50, 1], [700, 60, 16], 100), ((6, 3, 12), [20, 1], [40, 300], 0), ((2, 1, 80), [33], [33], 7), ((1, 1, 256), [1, 5], [640, 5], 0)])
def test_gates_per_feature_in_every_attention_kernel(dtype, sizes, q_lens, kv_lens, window):
    """Prompt tiles, tiles whose keys are cut in shares, single tokens with and without key ranges, the general kernel with and
    without: every one of them has its own last step, where the gates go."""
    from photon_infer_amd import ops
    H, G, d = sizes
    tdt, T, page = TORCH[dtype], sum(q_lens), 16
    rnd = lambda *s, seed: randn(*s, seed=seed).to(torch.bfloat16).double()
    q, gate = rnd(T, H, d, seed=1), randn(T, H * d + 8, seed=2, scale=2.0)
    k, v = [rnd(s, G, d, seed=10 + i) for i, s in enumerate(kv_lens)], [rnd(s, G, d, seed=20 + i) for i, s in enumerate(kv_lens)]
    scale = 0.7 / d ** 0.5
    want = gated_reference(q, k, v, q_lens, kv_lens, scale, window, gate[:, 8:])
    pool = PagedKV(list(zip([t.float() for t in k], [t.float() for t in v])), page, tdt, seed=4)
    ctx = attention_ctx(q_lens, kv_lens, tdt)
    out = torch.empty((T, H * d), dtype=tdt, device=DEV)
    ops.paged_attention(out, q.reshape(T, -1).to(tdt).to(DEV), pool.k, pool.v, pool.table, ctx, H, G, d, page, scale, window, None,
                        feature_gate=dev32(gate)[:, 8:])                 # a view of wider rows
    close(out, want, f"{sizes} {q_lens} of {kv_lens}", 3e-5 if dtype == "float32" else 1.2e-2)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("sizes", [(2, 1, 16, 8), (4, 2, 64, 16), (3, 3, 12, 6)])
@pytest.mark.parametrize("window", [1, 7, 16, 17, 33, 64])
def test_a_key_that_stands_out_is_seen_inside_the_window_only(dtype, sizes, window):
    """Query and key share one feature (outside the rotated ones) at a few loud positions, on and beside page borders; a token
    sees a loud key exactly while it is one of the ``window`` positions that end at itself - in prompts, in portions and alone."""
    from photon_infer_amd import ops
    H, G, d, rd = sizes
    T, page, tdt = 150, 16, TORCH[dtype]
    loud = [0, 15, 48, 100]
    k = torch.zeros(T, G, d, dtype=F64)
    k[:, :, d - 2] = 1.0
    k[loud] = 0.0
    k[loud, :, d - 1] = 3.0                                              # values are the keys as projected: 3 in the last feature
    q = torch.zeros(T, H, d, dtype=F64)
    q[:, :, d - 1] = 1.0
    proj = torch.cat([q.reshape(T, -1), k.reshape(T, -1), torch.full((T, H * d), 40.0, dtype=F64)], dim=1)
    table, pages = paged([T], page, seed=6)
    rotary = (dev32(30.0 ** (-2.0 * torch.arange(rd // 2, dtype=F64) / rd)), rd, False)
    for cuts in ([T], [16, 33, 2, 99], [40] + [1] * 110):
        kc, vc = torch.zeros((pages, G, page, d), dtype=tdt, device=DEV), torch.zeros((pages, G, d, page), dtype=tdt, device=DEV)
        outs, done = [], 0
        for n in cuts:
            ctx = attention_ctx([n], [done + n], tdt)
            qd = torch.empty((n, H * d), dtype=tdt, device=DEV)
            gates = ops.qk_rope_norm_write(qd, dev32(proj[done:done + n]), None, rotary, ctx, 1e-6, H, G, d, H * d, kc, vc, table, page)
            out = torch.empty((n, H * d), dtype=tdt, device=DEV)
            # both heads at root mean square 1: a loud pair scores scale * d
            ops.paged_attention(out, qd, kc, vc, table, ctx, H, G, d, page, 20.0 / d, window, None, feature_gate=gates)
            outs.append(out)
            done += n
        got = torch.cat(outs).double().cpu().view(T, H, d)[:, :, d - 1]
        for t in range(T):
            seen = any(0 <= t - p < window for p in loud)
            want = 3.0 if seen else 0.0
            assert float((got[t] - want).abs().max()) < 0.03, f"window {window} cuts {cuts[:3]} token {t}: {got[t].tolist()} instead of {want}"


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("sizes", [(4, 2, 16, 8, 7), (4, 1, 64, 64, 33), (6, 3, 12, 6, None), (1, 1, 96, 0, 1), (8, 2, 32, 16, 100), (2, 2, 80, 24, 40)])
def test_attention_part_whole_in_portions_and_token_by_token(dtype, sizes):
    from photon_infer_amd.config.llama import RopeScaling
    from photon_infer_amd.parts import POSITION_ENCODINGS
    H, G, d, rd, window = sizes
    D, T, page, scale, eps = 72, 150, 16, 1.7 / d ** 0.5, 1e-4
    tdt = TORCH[dtype]
    rnd = lambda *s, seed, scale=0.2: randn(*s, seed=seed, scale=scale).to(torch.bfloat16).double()
    W = {"q": rnd(H * d, D, seed=1), "k": rnd(G * d, D, seed=2), "g": rnd(H * d, D, seed=3), "o": rnd(D, H * d, seed=4),
         "q.b": rnd(H * d, seed=5, scale=0.5), "k.b": rnd(G * d, seed=6, scale=0.5)}
    h = randn(T, D, seed=12).to(tdt).double()
    m = {"heads": H, "kv_heads": G, "dim": d, "scale": scale, "mask": {"size": window} if window else None}
    rope = None
    if rd:
        m["rot"] = {"base": 300.0, "dims": rd, "scaling": {"factor": 4.0, "low": 1.0, "high": 4.0, "original": 128}}
        rope = POSITION_ENCODINGS.make("rope", head_dim=d, theta=300.0, rotary_dim=rd, scaling=RopeScaling("llama3", 4.0, 1.0, 4.0, 128))
        rope.load({}, tdt, torch.device(DEV))
    want = P.attention(h, m, W, "", eps, P.bf16_round if dtype == "bfloat16" else None)
    part = make_part("attention", W, tdt, hidden_size=D, num_heads=H, num_kv_heads=G, head_dim=d, position=rope, scale=scale, window=window,
                     names=("q", "k", "v", "o"), any_head_size=True, qkv_bias=True, accumulate=False, values_are_keys=True, head_norm_eps=eps, feature_gate="g")
    run_paged_part(part, h, want, ([T], [64, 7, 2, 77], [T - 12] + [1] * 12), tdt, page, 1e-4 if dtype == "float32" else 3e-2, f"{sizes}", D)


# ----------------------------------------------------------------------------- feed-forwards
@pytest.mark.parametrize("M,N,K", [(1, 40, 64), (5, 96, 2048), (200, 96, 128), (129, 520, 320), (300, 264, 1032), (520, 2048, 256), (3, 37, 90)])
def test_product_and_exact_gelu(M, N, K):
    """One token to many: the product's float32 result (or its pieces) through the activation's kernel, or the tile product's epilogue."""
    from photon_infer_amd import ops
    from photon_infer_amd.ops.workspace import KernelWorkspace
    a, w = randn(M, K, seed=1).to(torch.bfloat16), randn(N, K, seed=2, scale=3.0 / K ** 0.5).to(torch.bfloat16)
    want = P.gelu(a.double() @ w.double().T)
    assert float(want.min()) < -0.1 and float(want.max()) > 2.0
    ws = KernelWorkspace(DEV)
    for dtype in DTYPES:
        tdt = TORCH[dtype]
        out = torch.empty((M, N), dtype=tdt, device=DEV)
        ops.gemm_activation(out, a.to(tdt).to(DEV), w.to(tdt).to(DEV), "gelu", ws=ws)
        close(out, want, f"{dtype} {M} x {N} x {K}", 3e-5 if dtype == "float32" else 8e-3)


def test_gelu_epilogue_far_below_and_above_zero():
    """The tile product's epilogue has its own form of the error function: sums of exactly -12 .. 12 through it."""
    from photon_infer_amd import ops
    a = torch.zeros((256, 64))
    a[:, 0] = torch.linspace(-12, 12, 256)
    a = a.to(torch.bfloat16)
    w = torch.zeros((64, 64))
    w[:, 0] = 1.0
    out = torch.empty((256, 64), dtype=torch.bfloat16, device=DEV)
    ops.gemm_activation(out, a.to(DEV), w.to(torch.bfloat16).to(DEV), "gelu")
    want = torch.nn.functional.gelu(a[:, 0].double())
    got = out[:, 0].double().cpu()
    assert float((got - want).abs().max()) < 0.03 and float((got - want)[want.abs() < 1].abs().max()) < 3e-3
    assert float((got[want.abs() < 1e-3] - want[want.abs() < 1e-3]).abs().max()) < 1e-5


def test_routing_by_sigmoid_scores():
    from photon_infer_amd import ops
    T, E, top = 200, 11, 3
    z = randn(T, E, seed=1, scale=3.0)
    z[7, 4], z[7, 9] = 45.0, 50.0                     # both scores round to 1: the larger logit comes first all the same
    parts = randn(2, T, E, seed=3)
    for src in (dev32(z), ops.Partials(dev32(torch.cat([parts, (z - parts.sum(0))[None]])), 3, T, E)):
        ids, w = ops.route(src, top, scoring="sigmoid")
        for t in range(T):
            order, weights = P.route(z[t], top)
            assert ids[t].tolist() == order, t
            close(w[t], weights, f"weights of token {t}", 1e-5)
    assert ids[7, :2].tolist() == [9, 4]


@pytest.mark.parametrize("N,top,E,hi,tile", [(1, 1, 1, 1, 128), (7, 7, 3, 3, 64), (1000, 4, 16, 19, 128), (8192, 4, 16, 16, 128), (4096, 4, 16, 1, 128),
                                             (20000, 8, 128, 130, 64), (3000, 2, 1000, 1024, 128), (130, 2, 7, 7, 64)])
def test_entries_grouped_by_expert_in_order(N, top, E, hi, tile):
    from photon_infer_amd import ops
    ids = torch.randint(0, hi, (N // top, top), generator=torch.Generator().manual_seed(N), dtype=torch.int32)
    rows, flat = ops.group_entries(ids.to(DEV), E, tile), ids.view(-1).tolist()
    order = sorted((i for i in range(len(flat)) if flat[i] < E), key=lambda i: (flat[i], i))
    row_entry, entry_row = rows.row_entry.tolist(), rows.entry_row.tolist()
    assert row_entry[:len(order)] == order and not any(row_entry[len(order):])
    place = {e: k for k, e in enumerate(order)}
    assert entry_row == [place.get(i, 0) for i in range(len(flat))]
    want, row = [], 0
    for e in range(E):
        c = flat.count(e)
        want += [(e, row + k, min(tile, c - k)) for k in range(0, c, tile)]
        row += c
    got = list(zip(rows.tile_expert.tolist(), rows.tile_row0.tolist(), rows.tile_rows.tolist()))
    assert got[:len(want)] == want and all(t == (-1, 0, 0) for t in got[len(want):])


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("sizes", [(5, 2, 40, 0.5), (8, 4, 128, 1.5), (9, 1, 36, 0.3), (1, 1, 48, 0.7), (3, 3, 32, 2.0)])
@pytest.mark.parametrize("T", [1, 9, 150])
def test_routed_experts_weighed_on_their_input(dtype, sizes, T):
    from photon_infer_amd import ops
    from photon_infer_amd.parts import FEED_FORWARDS
    E, top, F, limit = sizes
    D, tdt = 64, TORCH[dtype]
    rnd = lambda *s, seed, scale=0.2: randn(*s, seed=seed, scale=scale).to(torch.bfloat16).double()
    W = {"router": rnd(E, D, seed=1, scale=0.3)}
    for e in range(E):
        W[f"e{e}.gate"], W[f"e{e}.up"], W[f"e{e}.down"] = rnd(F, D, seed=10 + e), rnd(F, D, seed=30 + e), rnd(D, F, seed=50 + e)
    part = FEED_FORWARDS.make("routed_experts", hidden_size=D, expert_size=F, num_experts=E, top=top, scoring="sigmoid", weigh_input=True,
                              activation="clamped_glu", limit=limit, alpha=P.GLU_ALPHA, accumulate=False)
    assert {s.name for s in part.tensor_specs()} == set(W)
    part.load({n: t.to(tdt).to(DEV) for n, t in W.items()}, tdt, torch.device(DEV))
    h = randn(T, D, seed=3).to(tdt).double()
    mlp = {"router": {"experts": E, "top": top}, "expert": {"ff": F, "limit": limit}}
    with RouteRecorder() as rec:
        out = torch.full((T, D), 7.0, device=DEV)
        part.forward(h.to(tdt).to(DEV), out, SimpleNamespace(workspace=None, may_defer=False))
    ids = rec.calls[0]
    margins, chosen = [], []
    P.routed_experts(h, mlp, W, "", margins=margins, chosen=chosen)
    for t in range(T):
        assert sorted(ids[t].tolist()) == sorted(chosen[t]) or (dtype == "bfloat16" and margins[t] < 0.02), (t, ids[t].tolist(), chosen[t], margins[t])
    want = P.routed_experts(h, mlp, W, "", P.bf16_round if dtype == "bfloat16" else None, choices=[r.tolist() for r in ids])
    close(out, want, f"{sizes} {T} tokens", 3e-5 if dtype == "float32" else 2e-2)
    clamped = sum(int(((P.sigmoid(h[t] @ W["router"][e]) * h[t] @ W[f"e{e}.up"].T).abs() > limit).sum()) for t in range(T) for e in ids[t].tolist())
    assert clamped > 0 or limit > 1.0                                  # the clamp is met


# ----------------------------------------------------------------------------- whole models
@pytest.fixture(scope="module")
def model_dirs(tmp_path_factory):
    root = tmp_path_factory.mktemp("semezen")
    return {name: TS.make_model_dir(root, name, seed=5) for name in TS.ALL}


_plain = {}
CLOSE_CALL = 0.05      # router logits: a bfloat16 choice that differs from the plain one must be this close to a tie


def plain_logits(model_dir, tokens, emulate=False, forced=None):
    key = (model_dir, tuple(tokens), emulate)
    if forced or key not in _plain:
        cfg, W = P.read_model_folder(model_dir)
        out = P.forward(cfg, W, list(tokens), P.bf16_round if emulate else None, choices=forced).float()
        if forced:
            return out
        _plain[key] = out
    return _plain[key]


def runner_for(model_dir, name, dtype, max_tokens):
    from photon_infer_amd.engine.replay import make_runner
    return make_runner(model_dir, dtype, max(max_tokens, 64), TS.ALL[name][1]["block_size"])


def check(got, model_dir, reqs, dtype, what, choices=None):
    """``choices`` (bfloat16 runs): the experts the engine chose per request; the plain logits are then those of the same choices,
    which must be the plain ones up to close calls."""
    assert got, "no logits came back"
    for rid, toks in reqs.items():
        forced = choices.get(rid) if choices else None
        if forced:
            cfg, W = P.read_model_folder(model_dir)
            margins, chosen = {}, {}
            P.forward(cfg, W, list(toks), P.bf16_round, choices=forced, margins=margins, chosen=chosen)
            for i, ids in forced.items():
                for t in range(len(toks)):
                    if sorted(ids[t]) != sorted(chosen[i][t]):
                        assert margins[i][t] < CLOSE_CALL, f"{what}: layer {i} token {t}: experts {ids[t]} instead of {chosen[i][t]} (margin {margins[i][t]:.4f})"
        ref = plain_logits(model_dir, toks, forced=forced)
        if dtype == "float32":
            tol = 1e-4 * max(1.0, float(ref.abs().max()))
        else:       # three times what rounding activations to bfloat16 does to the plain implementation itself
            tol = 3.0 * float((plain_logits(model_dir, toks, True, forced=forced) - ref).abs().max())
        for p in range(len(toks)):
            assert (rid, p) in got, f"{what}: logits of {rid} position {p} are missing"
            err = float((got[(rid, p)] - ref[p]).abs().max())
            assert err <= tol, f"{what}: {rid} position {p}: error {err:.3e} > {tol:.3e} (first wrong position)"


def run_checked(runner, steps, out_dir, model_dir, reqs, dtype, what):
    """Replay ``steps`` and compare; in bfloat16 the plain implementation follows the engine's routing choices."""
    if dtype == "float32":
        return check(run_trace(runner, steps, out_dir), model_dir, reqs, dtype, what)
    with RouteRecorder() as rec:
        got = run_trace(runner, steps, out_dir)
    check(got, model_dir, reqs, dtype, what, rec.by_request(steps, P.read_model_folder(model_dir)[0]))


LENGTHS = {"A": [1, 26, 90], "B": [3, 130, 210], "C": [2, 30, 75], "D": [2, 45, 100], "E": [1, 33, 70]}


def requests_for(name, seed=0):
    vocab = TS.ALL[name][0]["vocab"]
    return {f"r{i}": random_tokens(n, vocab, seed * 100 + i) for i, n in enumerate(LENGTHS[name])}


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(TS.ALL))
def test_whole_prompts_and_the_streams_after_every_layer(name, dtype, model_dirs, tmp_path):
    reqs = requests_for(name)
    steps = []
    for rid, toks in reqs.items():
        steps += cut_steps(rid, toks, [len(toks)], first_step=len(steps))
    runner = runner_for(model_dirs[name], name, dtype, live_token_need(steps))
    run_checked(runner, steps, str(tmp_path), model_dirs[name], reqs, dtype, "whole")
    if dtype == "float32":         # the sum of the streams after every layer; a layer's last update is left to the next reader
        from photon_infer_amd.engine.step import StepEntry
        from photon_infer_amd.parts.norm import LEFT_UPDATE
        toks = reqs["r2"]
        cfg, W = P.read_model_folder(model_dirs[name])
        want, got = [], []
        P.forward(cfg, W, toks, streams=want)
        n = cfg["streams"]
        for blk in runner.model.blocks:
            def wrapped(x, ctx, cache, f=blk.forward):
                f(x, ctx, cache)
                left, y, post = ctx.scratch[LEFT_UPDATE]
                assert left is x
                X, p = x.double().cpu(), post.double().cpu()
                got.append(sum(P.mix_streams([X[:, s] for s in range(n)], y.double().cpu(), p[n:].view(n, n), p[:n])))
            blk.forward = wrapped
        runner.admit("s")
        runner.step([StepEntry("s", toks, [])])
        assert len(got) == len(want) == len(cfg["layers"])
        for i, (g, w) in enumerate(zip(got, want)):
            close(g, w, f"streams after layer {i}", 1e-4)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(TS.ALL))
def test_prefill_then_token_by_token_and_all_token_by_token(name, dtype, model_dirs, tmp_path):
    reqs = requests_for(name, seed=1)
    steps = []
    for rid, toks in reqs.items():
        head = max(0, len(toks) - 40)
        steps += cut_steps(rid, toks, ([head] if head else []) + [1] * (len(toks) - head), first_step=len(steps))
    steps += cut_steps("all", reqs["r1"], [1], first_step=len(steps))
    runner = runner_for(model_dirs[name], name, dtype, live_token_need(steps))
    run_checked(runner, steps, str(tmp_path), model_dirs[name], dict(reqs, all=reqs["r1"]), dtype, "decoding")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(TS.ALL))
@pytest.mark.parametrize("sizes", [[2], [7, 2, 31, 1, 3], [64, 5], [17]])
def test_portions_of_changing_size(name, dtype, sizes, model_dirs, tmp_path):
    reqs = {"r2": requests_for(name, seed=2)["r2"]}
    steps = cut_steps("r2", reqs["r2"], sizes)
    runner = runner_for(model_dirs[name], name, dtype, live_token_need(steps))
    run_checked(runner, steps, str(tmp_path), model_dirs[name], reqs, dtype, f"portions {sizes}")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(TS.ALL))
def test_mixed_batches_with_pages_and_slots_used_again(name, dtype, model_dirs, tmp_path):
    """Seven unequal requests through four slots: some bring portions while others decode, and now and then single tokens
    only; a request may sit out a step; a finished request's pages and slot go to the next one.  Each must come out as it does alone."""
    vocab = TS.ALL[name][0]["vocab"]
    lengths = [70, 33, 5, 120, 64, 18, 91]
    reqs = {f"m{i}": random_tokens(n, vocab, 50 + i) for i, n in enumerate(lengths)}
    rng = np.random.default_rng(7)
    waiting, live, at, steps = list(reqs), [], {}, []
    while waiting or live:
        while waiting and len(live) < 4:
            live.append(waiting.pop(0))
            at[live[-1]] = 0
        entries, end, singles = [], [], rng.random() < 0.25
        for rid in list(live):
            left = len(reqs[rid]) - at[rid]
            if len(live) > 1 and rng.random() < 0.2:
                continue                               # sits this step out
            n = 1 if left <= 12 or singles else int(min(left - 12, rng.choice([2, 3, 16, 29, 40])))
            entries.append({"id": rid, "tokens": reqs[rid][at[rid]:at[rid] + n], "want": list(range(n))})
            at[rid] += n
            if at[rid] == len(reqs[rid]):
                end.append(rid)
                live.remove(rid)
        if entries:
            steps.append({"step": len(steps), "entries": entries, "end": end})
    runner = runner_for(model_dirs[name], name, dtype, live_token_need(steps))
    assert runner.cache.max_slots == 4
    run_checked(runner, steps, str(tmp_path), model_dirs[name], reqs, dtype, "mixed")
    assert all(g.pool.num_allocated == 0 for g in runner.cache.groups)


@pytest.mark.parametrize("dtype", DTYPES)
def test_a_long_prompt_whole_and_in_two_long_portions(dtype, model_dirs, tmp_path):
    vocab = TS.ALL["A"][0]["vocab"]
    reqs = {"w": random_tokens(600, vocab, 11), "p": random_tokens(600, vocab, 11)}
    steps = cut_steps("w", reqs["w"], [600])
    steps += cut_steps("p", reqs["p"], [301, 298, 1], first_step=len(steps))
    runner = runner_for(model_dirs["A"], "A", dtype, live_token_need(steps))
    run_checked(runner, steps, str(tmp_path), model_dirs["A"], reqs, dtype, "long prompt")


@pytest.mark.parametrize("name", ["A", "C", "D"])
def test_long_decoding_keeps_its_state(name, model_dirs, tmp_path):
    """250 tokens one by one after a portion of three: states and pages carry everything from step to step, windows give pages back."""
    vocab = TS.ALL[name][0]["vocab"]
    toks = random_tokens(250, vocab, 9)
    steps = cut_steps("long", toks, [3] + [1] * 247)
    runner = runner_for(model_dirs[name], name, "float32", 256)
    run_checked(runner, steps, str(tmp_path), model_dirs[name], {"long": toks}, "float32", "long decoding")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(TS.ALL))
def test_greedy_generation_through_the_engine(name, dtype, model_dirs):
    """The engine's own entry point, scheduler, sampling and decode steps: unequal prompts at once, more requests than slots,
    prompts longer than a portion; every request must generate what the plain implementation generates alone."""
    from photon_infer_amd.engine import ContinuousBatchEngine, EngineOptions
    cfg, W = P.read_model_folder(model_dirs[name])
    vocab = cfg["vocab"]
    prompts = [random_tokens(n, vocab, 70 + i) for i, n in enumerate([5, 41, 18, 70, 2])]
    engine = ContinuousBatchEngine(model_dirs[name], EngineOptions(dtype=dtype, block_size=TS.ALL[name][1]["block_size"], max_batch=3,
                                                                   max_cache_tokens=1024, chunk_size=32, max_model_len=200))
    got = engine.generate(prompts, max_new_tokens=10)
    for prompt, out in zip(prompts, got):
        want = P.greedy(cfg, W, prompt, 10)
        if dtype == "float32":
            assert list(out) == want
        else:       # bfloat16: a near tie may fall the other way; the differing token must be a close second of the plain logits
            for i, (a, b) in enumerate(zip(out, want)):
                if a != b:
                    lg = P.forward(cfg, W, prompt + want[:i])[-1]
                    tol = 3.0 * float((P.forward(cfg, W, prompt + want[:i], P.bf16_round)[-1] - lg).abs().max())
                    assert float(lg[b] - lg[a]) <= 2.0 * tol, f"token {i}: {a} instead of {b} ({float(lg[b] - lg[a]):.3f} apart, bound {tol:.3f})"
                    break


def test_command_line_and_replayed_decode_steps(model_dirs, tmp_path):
    """The framework's commands serve the design as they serve its others (from a folder, and from a bare configuration with
    random weights); and decode steps replayed as HIP graphs give the tokens of eager steps, with new requests' prompts in
    between and states in slots that are used again."""
    import subprocess
    from photon_infer_amd.engine import ContinuousBatchEngine, EngineOptions
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    cfg, W = P.read_model_folder(model_dirs["A"])
    prompt = random_tokens(9, cfg["vocab"], 81)
    want = P.greedy(cfg, W, prompt, 5)
    proc = subprocess.run([os.path.join(root, "bin", "llama_infer"), model_dirs["A"], "--dtype", "fp32", "--prompt-ids",
                           ",".join(map(str, prompt)), "--max-new-tokens", "5", "--temperature", "0", "--ignore-eos"],
                          capture_output=True, text=True, timeout=300)
    assert proc.returncode == 0, proc.stderr[-2000:]
    assert "Architecture: Semezen" in proc.stdout and f"Generated ids: {','.join(map(str, want))}" in proc.stdout
    (tmp_path / "cfg").mkdir()
    json.dump(TS.TINY_E, open(tmp_path / "cfg" / "config.json", "w"))
    proc = subprocess.run([os.path.join(root, "bin", "llama_infer"), str(tmp_path / "cfg"), "--random-weights", "--seed", "3",
                           "--prompt-ids", "5,6,7", "--max-new-tokens", "4", "--ignore-eos"], capture_output=True, text=True, timeout=300)
    assert proc.returncode == 0, proc.stderr[-2000:]
    assert "Generated ids:" in proc.stdout
    cfgc, _ = P.read_model_folder(model_dirs["C"])
    toks = random_tokens(12, cfgc["vocab"], 82)
    lines = "\n".join(json.dumps(s) for s in cut_steps("x", toks, [5, 1, 6])) + "\n"
    proc = subprocess.run([os.path.join(root, "bin", "trace_run"), "--model", model_dirs["C"], "--dtype", "float32", "--out", str(tmp_path / "out"),
                           "--max-tokens", "64"], input=lines, capture_output=True, text=True, timeout=300)
    assert proc.returncode == 0, proc.stderr[-2000:]
    assert [l for l in proc.stdout.split("\n") if l.startswith("done")] == ["done 0", "done 1", "done 2"]
    last = torch.from_numpy(np.fromfile(tmp_path / "out" / "2.f32", dtype="<f4").reshape(6, cfgc["vocab"]))
    close(last, plain_logits(model_dirs["C"], toks)[6:].double(), "trace_run", 1e-4)

    prompts = [random_tokens(n, cfg["vocab"], 90 + n) for n in (3, 40, 17, 9, 26)]

    def run(use_graphs):
        eng = ContinuousBatchEngine(model_dirs["A"], EngineOptions(dtype="bfloat16", block_size=16, max_batch=3, max_cache_tokens=1024,
                                                                   chunk_size=8, max_step_tokens=24, max_model_len=200, use_graphs=use_graphs))
        assert eng.runner.graph_safe
        out = eng.generate(prompts, max_new_tokens=20, ignore_eos=True)
        return out, eng.runner.graphs_captured

    graphs, captured = run(True)
    eager, none = run(False)
    assert captured > 0 and none == 0
    assert [list(o) for o in graphs] == [list(o) for o in eager]


def wide_config():
    attn = dict(heads=16, kv_heads=4, dim=64, vdim=64, scale=0.12, mask={"size": 150},
                rot={"base": 10000.0, "dims": 32, "scaling": {"factor": 4.0, "low": 1.0, "high": 4.0, "original": 256}})
    moe = {"kind": "moe", "expert": {"ff": 512, "limit": 1.5}, "router": {"experts": 8, "top": 3}}
    return {"architecture": "Semezen", "vocab": 1000, "width": 1024, "streams": 4, "norm": {"eps": 1e-5},
            "layers": [{"type": "mingru", "mixer": {"width": 1024}, "mlp": {"kind": "dense", "ff": 3072}}, {"type": "attention", "mixer": attn, "mlp": moe},
                       {"type": "mingru", "mixer": {"width": 512}, "mlp": moe}, {"type": "attention", "mixer": attn, "mlp": {"kind": "dense", "ff": 2048}}]}


def test_kernels_chosen_at_real_widths_against_the_general_kernels(tmp_path):
    """A model wide enough that the bfloat16 engine takes what it takes at real sizes (tile products with their epilogues for the
    prompt, weight-streaming products left in pieces for single tokens, the matrix-core attention, grouped tile products) against
    the same engine on the general kernels: a 300-token prompt, a mixed step and decode steps of a batch, the same experts in both."""
    from photon_infer_amd import ops
    from photon_infer_amd.config import SemezenConfig
    from photon_infer_amd.engine.replay import make_runner
    from photon_infer_amd.engine.step import StepEntry
    from photon_infer_amd.weights import write_random_model
    d = write_random_model(SemezenConfig.from_dict(wide_config()), str(tmp_path / "wide"), seed=2, std=0.03, norm_init="uniform", dtype="bfloat16")
    prompts = {"a": random_tokens(300, 1000, 1), "b": random_tokens(70, 1000, 2), "c": random_tokens(5, 1000, 3)}
    outs, routes = [], []
    real = ops.route
    for fast in (True, False):
        prev = ops.use_fast_kernels(fast)
        calls = []

        def route(*a, **k):
            ids, w = real(*a, **k)
            if fast:
                routes.append(ids)
                return ids, w
            forced = routes[len(calls)]                # the second run follows the first run's experts
            calls.append(1)
            return forced, torch.sigmoid(a[0]).gather(1, forced.long()).contiguous()
        ops.route = route
        try:
            r = make_runner(d, "bfloat16", 1024, 16)
            for rid in prompts:
                r.admit(rid)
            got = [r.step([StepEntry("a", prompts["a"], [0, 150, 299])]),
                   r.step([StepEntry("b", prompts["b"][:60], [59]), StepEntry("c", prompts["c"], [4]), StepEntry("a", [7], [0])])]
            for k in range(3):
                got.append(r.step([StepEntry("a", [8 + k], [0]), StepEntry("b", [prompts["b"][60 + k]], [0]), StepEntry("c", [9 + k], [0])]))
            outs.append(torch.cat(got).float().cpu())
            if fast:
                assert r.workspace.counts["added_by_streams"] > 0
        finally:
            ops.route = real
            ops.use_fast_kernels(prev)
    err = float((outs[0] - outs[1]).abs().max())
    assert err <= 0.04 * float(outs[1].std()) + 0.02, (err, float(outs[1].std()))
