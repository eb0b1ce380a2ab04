"""Roserax on the GPU against the plain implementation (``plain_roserax``): each mechanism's kernels alone, with inputs made so
that a fault shows (keys that stand out just inside and just outside a window and among and behind the kept first tokens, a
write that must be recalled after hundreds of tokens, a loud latent far back), then whole models under every cutting,
batching, page and slot reuse, long decoding, and greedy generation through the engine's own entry point."""
import json
import math
import os
from types import SimpleNamespace

import numpy as np
import pytest
import torch

import plain_roserax as P
import tiny_roserax as TR
from gpu_tools import (DEV, PagedKV, RouteRecorder, attention_ctx, close, cut_steps, dev32, in_steps, live_token_need, make_part, paged, randn,
                       run_paged_part, run_trace, state_ctx)
from tiny_models import random_tokens

pytestmark = pytest.mark.gpu
DTYPES = ["float32", "bfloat16"]
TORCH = {"float32": torch.float32, "bfloat16": torch.bfloat16}
F64 = torch.float64


def act_tol(dtype):
    return 3e-5 if dtype == "float32" else 1.2e-2


# ----------------------------------------------------------------------------- a window that keeps the first tokens
def kept_attend(q, k, v, scale, size, keep):
    T, H, G = q.shape[0], q.shape[1], k.shape[1]
    seen = P.kept_window_mask(T, size, keep)
    out = torch.zeros((T, H, v.shape[2]), dtype=F64)
    for n in range(H):
        g = n // (H // G)
        out[:, n] = P.softmax_over((q[:, n] @ k[:, g].T) * scale, seen, one=True) @ v[:, g]
    return out


# heads, kv heads, key width, value width, window, kept: both sides of pages (16), chunks (32) and rounds (64, 128) of keys
KEPT = [(4, 2, 16, 32, 24, 5), (4, 1, 64, 64, 33, 16), (6, 3, 24, 12, 7, 11), (2, 2, 128, 128, 100, 17), (3, 3, 40, 40, 1, 1), (8, 2, 48, 48, 64, 31),
        (4, 4, 64, 64, 130, 33), (16, 2, 32, 32, 40, 70), (2, 1, 160, 160, 50, 130), (1, 1, 80, 80, 20, 1), (20, 1, 64, 64, 65, 6), (4, 2, 256, 256, 30, 40),
        (2, 2, 64, 64, 500, 9), (2, 1, 64, 64, 90, 129)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("sizes", KEPT)
def test_window_with_kept_tokens_and_a_one_in_the_denominator(dtype, sizes):
    """A whole prompt, then its last tokens alone and in portions, over pages dealt out of order, the pages between the kept
    tokens and the window given back.  The last query is loud towards four keys: the last kept one and the window's first one
    (seen), the one behind the kept ones and the one in front of the window (not seen, and louder)."""
    from photon_infer_amd import ops
    H, G, d, dv, size, keep = sizes
    T, page, scale = 333, 16, 0.3
    tdt = TORCH[dtype]
    q, k, v = randn(T, H, d, seed=1), randn(T, G, d, seed=2), randn(T, G, dv, seed=3)
    mark, lo = randn(d, seed=9) * (16.0 / d) ** 0.5, max(0, T - size)
    q[-1] = mark * 1.5
    inside, outside = {keep - 1, lo}, {j for j in (keep, lo - 1) if keep <= j < lo}
    for n, j in enumerate(sorted(inside)):
        k[j], v[j] = mark * (1.0 + 0.05 * n), v[j] + 4.0 * (n + 1)
    for j in outside:
        k[j], v[j] = mark * 1.3, v[j] - 9.0
    rnd = lambda t: t.to(tdt).double()
    want = kept_attend(rnd(q), rnd(k), rnd(v), scale, size, keep)
    if outside:      # a mask that is one key off on any side is another result
        for other in ((size + 1, keep), (max(1, size - 1), keep), (size, keep + 1), (size, keep - 1)):
            if other[0] != size or min(keep, other[1]) < lo:
                off = kept_attend(rnd(q[-1:]).expand(T, -1, -1), rnd(k), rnd(v), scale, *other)
                if size > 1 or other[0] > size:
                    assert float((want[-1] - off[-1]).abs().max()) > 0.1, other
    kv = PagedKV([(k, v)], page, tdt, seed=3)
    ones = torch.zeros(H, device=DEV)
    tol = 3e-5 if dtype == "float32" else 3e-2
    for q_len in (T, 1, 4, 70, 2):
        table = kv.table.clone()
        first = T - q_len                                  # nothing a later query needs is missing, everything else is
        gone = range(-(-keep // page), max(0, first - size + 1) // page)
        for b in gone:
            table[0, b] = -1
        ctx = attention_ctx([q_len], [T], tdt)
        rows = slice(T - q_len, T)
        qd = q[rows].reshape(q_len, -1).to(tdt).to(DEV).contiguous()
        out = torch.empty((q_len, H * dv), dtype=tdt, device=DEV)
        ops.paged_attention(out, qd, kv.k, kv.v, table, ctx, H, G, d, page, scale, size, None, value_dim=dv, sinks=ones, keep_first=keep)
        close(out, want[rows].reshape(q_len, -1), f"{sizes} {q_len} tokens ending the sequence", tol)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("sizes", [(4, 2, 64, 64, 40, 20), (8, 1, 32, 32, 150, 140), (3, 3, 20, 12, 30, 9)])
def test_long_contexts_in_key_ranges_and_cut_tiles(dtype, sizes):
    """Single tokens and portions late in long contexts of several requests at once: the keys are walked in ranges (and a tile's in
    shares) that lie in the kept tokens, in the window or across both; and a batch of single tokens and portions together."""
    from photon_infer_amd import ops
    H, G, d, dv, size, keep = sizes
    page, scale, tdt = 16, 0.25, TORCH[dtype]
    lens = [1500, 37, 701, 64]
    seqs, wants = [], []
    for r, n in enumerate(lens):
        q, k, v = randn(n, H, d, seed=10 + r), randn(n, G, d, seed=20 + r), randn(n, G, dv, seed=30 + r)
        v[:keep] += 3.0                                    # the kept tokens show in every result
        seqs.append((q, k, v))
        rnd = lambda t: t.to(tdt).double()
        tail = range(max(0, n - 64), n)
        w = {}
        for i in tail:
            seen = [j for j in range(i + 1) if i - j < size or j < keep]
            o = torch.zeros((H, dv), dtype=F64)
            for h in range(H):
                s = rnd(k)[seen, h // (H // G)] @ rnd(q)[i, h] * scale
                p = P.softmax_over(s[None], torch.ones((1, len(seen)), dtype=torch.bool), one=True)[0]
                o[h] = p @ rnd(v)[seen, h // (H // G)]
            w[i] = o.reshape(-1)
        wants.append(w)
    kv = PagedKV([(k, v) for _, k, v in seqs], page, tdt, seed=4)
    ones, tol = torch.zeros(H, device=DEV), 3e-5 if dtype == "float32" else 3e-2
    for q_lens in ([1, 1, 1, 1], [64, 1, 40, 2], [3, 37, 1, 64]):
        ctx = attention_ctx(q_lens, lens, tdt)
        qd = torch.cat([q[n - m:].reshape(m, -1) for (q, _, _), n, m in zip(seqs, lens, q_lens)]).to(tdt).to(DEV).contiguous()
        out = torch.empty((sum(q_lens), H * dv), dtype=tdt, device=DEV)
        ops.paged_attention(out, qd, kv.k, kv.v, kv.table, ctx, H, G, d, page, scale, size, None, value_dim=dv, sinks=ones, keep_first=keep)
        want = torch.stack([wants[r][i] for r, (n, m) in enumerate(zip(lens, q_lens)) for i in range(n - m, n)])
        close(out, want, f"{sizes} {q_lens}", tol)


def test_kept_tokens_need_no_other_option():
    """keep_first alone (no sink): an ordinary softmax over the kept keys and the window."""
    from photon_infer_amd import ops
    T, H, d, size, keep, page = 200, 4, 64, 20, 10, 16
    for tdt in (torch.float32, torch.bfloat16):
        q, k, v = (randn(T, H, d, seed=s).to(tdt).double() for s in (1, 2, 3))
        seen = P.kept_window_mask(T, size, keep)
        want = torch.stack([P.softmax_over(q[:, n] @ k[:, n].T * 0.2, seen, one=False) @ v[:, n] for n in range(H)], dim=1)
        kv = PagedKV([(k, v)], page, tdt)
        for n in (T, 1):
            out = torch.empty((n, H * d), dtype=tdt, device=DEV)
            ops.paged_attention(out, q[T - n:].reshape(n, -1).to(tdt).to(DEV), kv.k, kv.v, kv.table, attention_ctx([n], [T], tdt), H, H, d, page, 0.2, size,
                                None, keep_first=keep)
            close(out, want[T - n:].reshape(n, -1), f"{tdt} {n}", 3e-5 if tdt == torch.float32 else 3e-2)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("sizes", [(4, 2, 16, 32, 0), (4, 1, 64, 64, 32), (6, 3, 24, 12, 24), (3, 3, 10, 7, 4), (1, 1, 48, 80, 0), (2, 1, 320, 40, 6), (8, 4, 128, 128, 0)])
@pytest.mark.parametrize("T", [1, 45])
@pytest.mark.parametrize("splits", [0, 3, 9])
def test_heads_normalised_with_one_weight_and_values_of_their_own(dtype, sizes, T, splits):
    """Rotation (or none), norm per head with a weight for all heads, keys and values into pages, gates as they are; from a tensor
    and from pieces.  One loud head must not change its neighbours' norms."""
    from photon_infer_amd import ops
    from photon_infer_amd.ops.workspace import Partials
    H, G, d, dv, rd = sizes
    page, eps, tdt, ng = 8, 3e-3, TORCH[dtype], 12
    N = (H + G) * d + G * dv + ng
    row = randn(T, N, seed=4, scale=2.0)
    row[:, :d] *= 30.0
    wq, wk = 0.5 + torch.rand(d, dtype=F64), 0.5 + torch.rand(d, dtype=F64)
    table, pages = paged([T], page)
    kc = torch.zeros((pages, G, page, d), dtype=tdt, device=DEV)
    vc = torch.zeros((pages, G, dv, page), dtype=tdt, device=DEV)
    ctx = attention_ctx([T], [T], tdt)
    freqs = torch.tensor([200.0 ** (-2.0 * i / max(rd, 1)) for i in range(rd // 2)], dtype=torch.float32, device=DEV)
    if splits:
        pieces = torch.cat([randn(splits - 1, T, N, seed=5), torch.zeros(1, T, N, dtype=F64)])
        pieces[-1] = row - pieces.sum(0)
        proj = Partials(dev32(pieces), splits, T, N)
        row = proj.part.double().cpu().sum(0)
    else:
        proj = dev32(row)
        row = proj.double().cpu()
    q = torch.empty((T, H * d), dtype=tdt, device=DEV)
    gates = ops.qk_rope_norm_write(q, proj, None, (freqs, rd, False) if rd else None, ctx, eps, H, G, d, ng, kc, vc, table, page, value_dim=dv,
                                   w_q=dev32(wq), w_k=dev32(wk))
    pos = torch.arange(T)
    turned = lambda t: P.rotate_halves(t, pos, rd, 200.0) if rd else t
    tol = 1e-5 if dtype == "float32" else 1e-2
    close(q, P.rms_norm(turned(row[:, :H * d].reshape(T, H, d)), wq, eps).reshape(T, -1), "queries", tol)
    close(gates, row[:, -ng:], "gates", 1e-5)
    want_k = P.rms_norm(turned(row[:, H * d:(H + G) * d].reshape(T, G, d)), wk, eps)
    want_v = row[:, (H + G) * d:N - ng].reshape(T, G, dv)
    for t in sorted({0, T // 2, T - 1}):
        pg, slot = int(table[0, t // page]), t % page
        close(kc[pg, :, slot], want_k[t], f"key {t} in its page", tol)
        close(vc[pg, :, :, slot], want_v[t], f"value {t} in its page", tol)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("sizes", [(4, 2, 16, 32, 24, 5), (3, 3, 20, 12, 9, 20), (4, 1, 64, 64, 50, 17), (2, 1, 48, 48, None, 0)])
def test_attention_mixer_as_a_part(dtype, sizes):
    H, G, d, dv, size, keep = sizes
    D, T, eps, tdt = 72, 130, 1e-4, TORCH[dtype]
    m = {"heads": H, "kv_heads": G, "dim": d, "vdim": dv, "scale": 0.4, "mask": {"size": size, "keep_first": keep} if size else None}
    shapes = {"q": (H * d, D), "k": (G * d, D), "v": (G * dv, D), "o": (D, H * dv)}
    W = {n: randn(*s, seed=10 + i, scale=0.2).to(torch.bfloat16).double() for i, (n, s) in enumerate(shapes.items())}
    W["q.norm"], W["k.norm"] = 0.5 + torch.rand(d, dtype=F64), 0.5 + torch.rand(d, dtype=F64)
    part = make_part("sink_window_attention", W, tdt, hidden_size=D, num_heads=H, num_kv_heads=G, head_dim=d, value_dim=dv, scale=0.4, window=size,
                     keep_first=keep, eps=eps, norm_per_head=True, norm_shared=True, distance_bias=False, sink_score=0.0, output_gate=False, accumulate=False)
    h = randn(T, D, seed=3).to(tdt).double()
    want = P.window_attention(h, m, W, eps)
    run_paged_part(part, h, want, ([T], [64, 7, 2, 57], [T - 12] + [1] * 12), tdt, 16, 1e-4 if dtype == "float32" else 4e-2, f"{sizes}", D)


# ----------------------------------------------------------------------------- attention through a latent, with gates
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("sizes", [(2, 16, 8, 24, 20, 24), (4, 32, 16, 32, 64, 48), (3, 20, 6, 28, 10, 30), (1, 24, 16, 40, 32, 272), (5, 8, 2, 8, 8, 8),
                                   (20, 8, 8, 8, 16, 24), (16, 16, 16, 16, 32, 112)])
def test_gated_latent_mixer_whole_in_portions_and_token_by_token(dtype, sizes):
    """Halves paired in the rotation, a gate per feature; one latent far back is loud.  Whole prompts longer than 128 tokens take the
    grouped tile kernel's gated epilogue in bfloat16."""
    H, d, dr, dv, qr, rank = sizes
    D, T, eps, base, tdt = 72, 150, 1e-5, 300.0, TORCH[dtype]
    m = {"heads": H, "dim": d, "rot_dim": dr, "vdim": dv, "q_rank": qr, "kv_rank": rank, "scale": 0.15, "rot": {"base": base, "dims": dr}}
    shapes = {"dq": (qr, D), "uq": (H * (d + dr), qr), "dkv": (rank + dr, D), "uk": (H * d, rank), "uv": (H * dv, rank), "o": (D, H * dv), "g": (H * dv, D)}
    W = {n: randn(*s, seed=10 + i, scale=0.2).to(torch.bfloat16).double() for i, (n, s) in enumerate(shapes.items())}
    W["dq.norm"], W["dkv.norm"] = 0.5 + torch.rand(qr, dtype=F64), 0.5 + torch.rand(rank, dtype=F64)
    h = randn(T, D, seed=3).to(tdt).double()
    h[5] *= 4.0
    want = P.latent_attention(h, m, W, eps)
    from photon_infer_amd.parts import POSITION_ENCODINGS
    rope = POSITION_ENCODINGS.make("rope", head_dim=dr, theta=base)
    part = make_part("latent_attention", W, tdt, hidden_size=D, num_heads=H, head_dim=d, rot_dim=dr, value_dim=dv, q_rank=qr, kv_rank=rank, scale=0.15,
                     eps=eps, position=rope, gate="g", accumulate=False)
    run_paged_part(part, h, want, ([T], [64, 7, 2, 77], [T - 12] + [1] * 12), tdt, 16, 1e-4 if dtype == "float32" else 4e-2, f"{sizes}", D)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("sizes", [(1, 3, 24, 30), (9, 4, 16, 24), (77, 2, 128, 200), (8, 5, 7, 65), (300, 3, 64, 96), (257, 4, 40, 72), (140, 2, 256, 130)])
def test_a_product_per_head_with_gates(dtype, sizes):
    from photon_infer_amd import ops
    M, H, K, N = sizes
    tdt = TORCH[dtype]
    a, w, z = randn(M, H * K, seed=1).to(tdt), randn(H, K, N, seed=2).to(tdt), randn(M, H * N + 5, seed=3, scale=3.0)
    want = torch.einsum("mhk,hkn->mhn", a.double().reshape(M, H, K), w.double()).reshape(M, -1) * P.sigmoid(z[:, :H * N])
    out = torch.full((M, H * N), 7.0, dtype=tdt, device=DEV)
    rows = w.transpose(1, 2).contiguous().to(DEV) if dtype == "bfloat16" else None
    ops.head_gemm(out, a.to(DEV), w.to(DEV).contiguous(), H, w_rows=rows, gate=dev32(z))
    close(out, want, f"{sizes}", 2e-5 if dtype == "float32" else 2e-2)


# ----------------------------------------------------------------------------- retention
def retention_case(T, H, d, dv, rd, interleaved=False, seed=1):
    proj = randn(T, 2 * H * (d + dv), seed=seed)
    q, k = proj[:, :H * d].reshape(T, H, d), proj[:, H * d:2 * H * d].reshape(T, H, d)
    v, g = proj[:, 2 * H * d:2 * H * d + H * dv].reshape(T, H, dv), proj[:, 2 * H * d + H * dv:]
    return proj, q, k, v, g


def turned(x, positions, rd, base, interleaved):
    if not rd:
        return x
    if interleaved:      # neighbours: the same rotation on the features in another order
        order = torch.arange(rd).view(rd // 2, 2).t().reshape(-1)
        y = x.clone()
        y[..., order] = P.rotate_halves(x[..., order], positions, rd, base)
        return y
    return P.rotate_halves(x, positions, rd, base)


RET = [(2, 16, 24, 16, False), (1, 10, 7, 6, False), (3, 64, 32, 32, False), (2, 128, 128, 128, False), (2, 36, 20, 36, False), (1, 96, 200, 12, True),
       (2, 72, 300, 40, False), (1, 256, 64, 256, False), (4, 8, 8, 0, False), (1, 130, 516, 20, False), (2, 20, 256, 10, True)]
RET_CUTS = ({"a": [150], "b": [9], "c": [1]}, {"a": [1], "b": [1], "c": [1]}, {"a": [2, 63, 1, 65, 17], "b": [3, 2], "c": [1]}, {"a": [64], "b": [1, 8], "c": [1]},
            {"a": [149, 1], "b": [8, 1], "c": [1]})


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("sizes", RET)
def test_retention_under_every_cutting(dtype, sizes):
    """Three requests at once, whole, token by token, in portions on both sides of a chunk of 64; states in slots dealt out of order."""
    from photon_infer_amd import ops
    H, d, dv, rd, inter = sizes
    eps, base = 1e-4, 90.0
    lens = {"a": 150, "b": 9, "c": 1}
    slot = {"a": 3, "b": 0, "c": 2}
    decay = [0.3, 0.97, 1.0, 0.999][:H]
    case = {n: retention_case(T, H, d, dv, rd, seed=7 * i + 1) for i, (n, T) in enumerate(lens.items())}
    want, states = {}, {}
    for n, (proj, q, k, v, g) in case.items():
        pos = torch.arange(lens[n])
        o, states[n] = P.retention_heads(turned(q, pos, rd, base, inter), turned(k, pos, rd, base, inter) * d ** -0.5, v, decay)
        want[n] = P.rms_norm(o, None, eps).reshape(lens[n], -1) * P.silu(g)
    freqs = torch.tensor([base ** (-2.0 * i / max(rd, 1)) for i in range(rd // 2)], dtype=torch.float32, device=DEV)
    table = ops.decay_table(decay, DEV)
    for cuts in RET_CUTS:
        state = torch.full((4, H * d * dv), 5.0, device=DEV)
        for n in lens:
            state[slot[n]] = 0.0
        for step in in_steps(lens, cuts):
            ctx = state_ctx([e - b for _, b, e in step], [slot[n] for n, _, _ in step])
            ctx.all_decode = all(e - b == 1 for _, b, e in step)
            ctx.positions = torch.cat([torch.arange(b, e, dtype=torch.int32) for _, b, e in step]).to(DEV)
            proj = dev32(torch.cat([case[n][0][b:e] for n, b, e in step]))
            y = torch.empty((ctx.T, H * dv), dtype=TORCH[dtype], device=DEV)
            ops.retention(y, proj, (freqs, rd, inter) if rd else None, table, d ** -0.5, eps, ctx, state, H, d, dv)
            at = 0
            for n, b, e in step:
                close(y[at:at + e - b], want[n][b:e], f"{sizes} {cuts['a'][:3]} {n} {b}..{e}", 1e-4 if dtype == "float32" else 1.2e-2)
                at += e - b
        for n in lens:
            close(state[slot[n]].view(H, d, dv), states[n], f"state of {n}", 3e-5)
        assert bool((state[1] == 5.0).all())


@pytest.mark.parametrize("splits", [2, 9])
def test_retention_of_single_tokens_adds_pieces(splits):
    from photon_infer_amd import ops
    from photon_infer_amd.ops.workspace import Partials
    H, d, dv, R, eps, base = 2, 32, 48, 3, 1e-4, 50.0
    N = 2 * H * (d + dv)
    pieces, S0 = randn(splits, R, N, seed=1), randn(R, H, d, dv, seed=2)
    row = pieces.sum(0)
    pos, decay = torch.tensor([5, 0, 77]), [0.9, 0.99]
    q, k = (P.rotate_halves(row[:, i * H * d:(i + 1) * H * d].reshape(R, H, d), pos, d, base) for i in (0, 1))
    v = row[:, 2 * H * d:2 * H * d + H * dv].reshape(R, H, dv)
    want = torch.cat([P.rms_norm(P.retention_heads(q[r:r + 1], k[r:r + 1] * d ** -0.5, v[r:r + 1], decay, S0[r])[0], None, eps).reshape(1, -1) for r in range(R)])
    want = want * P.silu(row[:, 2 * H * d + H * dv:])
    state = dev32(S0.reshape(R, -1)[[2, 0, 1]])
    ctx = state_ctx([1] * R, [1, 2, 0])
    ctx.all_decode, ctx.positions = True, pos.to(torch.int32).to(DEV)
    freqs = torch.tensor([base ** (-2.0 * i / d) for i in range(d // 2)], dtype=torch.float32, device=DEV)
    y = torch.empty((R, H * dv), device=DEV)
    ops.retention(y, Partials(dev32(pieces), splits, R, N), (freqs, d, False), ops.decay_table(decay, DEV), d ** -0.5, eps, ctx, state, H, d, dv)
    close(y, want, "single tokens from pieces", 1e-4)


@pytest.mark.parametrize("cuts", [[2000], [1] * 3 + [997, 1000], [640] * 3 + [80], [17] * 118])
def test_a_write_recalled_a_thousand_tokens_later(cuts):
    """One key that nothing else resembles: without a decay what it wrote comes back whole after 1,900 tokens, with a decay it comes
    back as the power of the distance says, and another head's decay of zero leaves nothing."""
    from photon_infer_amd import ops
    H, d, dv, T, at = 3, 8, 8, 2000, 37
    decay = [1.0, 0.9995, 0.0]
    proj = torch.zeros(T, 2 * H * (d + dv), dtype=F64)
    for h in range(H):
        proj[at, H * d + h * d + 3] = 1.0                                             # the key
        proj[at, 2 * H * d + h * dv:2 * H * d + (h + 1) * dv] = torch.arange(1.0, 9.0)   # what it writes
        proj[at + 1:, h * d + 3] = 1.0                                                # everybody behind asks for it
    proj[:, 2 * H * d + H * dv:] = 20.0                                               # open gates
    state = torch.zeros(1, H * d * dv, device=DEV)
    got, done = [], 0
    for n in cuts:
        n = min(n, T - done)
        if n == 0:
            break
        ctx = state_ctx([n], [0])
        ctx.all_decode, ctx.positions = n == 1, torch.arange(done, done + n, dtype=torch.int32, device=DEV)
        y = torch.empty((n, H * dv), device=DEV)
        ops.retention(y, dev32(proj[done:done + n]), None, ops.decay_table(decay, DEV), 1.0, 1.0, ctx, state, H, d, dv)
        got.append(y)
        done += n
    y = torch.cat(got).double().cpu() / 20.0
    for t in (at + 1, 100, 1000, T - 1):
        for h in range(H):
            o = torch.arange(1.0, 9.0, dtype=F64) * decay[h] ** (t - at)
            close(y[t, h * dv:(h + 1) * dv], P.rms_norm(o, None, 1.0), f"head {h} token {t}", 2e-4)
    assert bool((y[:at] == 0).all())


def test_retention_decays_must_fit():
    from photon_infer_amd.errors import UnsupportedModelError
    from photon_infer_amd.parts import MIXERS
    for bad in ([0.5], [0.5, 1.01], [-0.1, 0.5]):
        with pytest.raises(UnsupportedModelError, match="decays"):
            MIXERS.make("retention", hidden_size=8, num_heads=2, key_dim=4, value_dim=4, decays=bad, eps=1e-5)


# ----------------------------------------------------------------------------- a result between two norms
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("T,D", [(7, 64), (5, 90), (600, 256), (4, 2048), (3, 4100), (2, 12288), (6, 33), (700, 3072)])
def test_a_result_joins_the_stream_between_two_norms(dtype, T, D):
    from photon_infer_amd import ops
    x, y, post, nxt = randn(T, D, seed=1, scale=2.0), randn(T, D, seed=2), randn(D, seed=3) * 0.3 + 1.0, randn(D, seed=4) * 0.3 + 1.0
    new = x + P.rms_norm(y, post, 1e-3)
    h = P.rms_norm(new, nxt, 2e-2)
    kw = dict(nxt=dev32(nxt), next_eps=2e-2, h_dtype=TORCH[dtype])
    X = dev32(x)
    close(ops.rms_join(X, dev32(y), dev32(post), 1e-3, **kw), h, "h", act_tol(dtype))
    close(X, new, "stream")
    X = dev32(x)
    assert ops.rms_join(X, dev32(y), dev32(post), 1e-3) is None
    close(X, new, "update alone")
    rows = torch.tensor([T - 1, 0, T // 2], dtype=torch.int32, device=DEV)
    X = dev32(x)
    close(ops.rms_join(X, dev32(y), dev32(post), 1e-3, rows=rows, **kw), h[rows.cpu().long()], "chosen rows", act_tol(dtype))
    close(X, x, "chosen rows leave the stream", 1e-6)


@pytest.mark.parametrize("D", [640, 90])
@pytest.mark.parametrize("splits", [2, 8, 11])
def test_joining_adds_the_pieces_of_a_result(D, splits):
    from photon_infer_amd import ops
    from photon_infer_amd.ops.workspace import KernelWorkspace, Partials, PendingUpdate
    T = 5
    x, pieces, post, nxt = randn(T, D, seed=1), randn(splits, T, D, seed=2), randn(D, seed=3), randn(D, seed=4)
    new = x + P.rms_norm(pieces.sum(0), post, 1e-4)
    ws = KernelWorkspace(DEV)
    y = torch.full((T, D), float("nan"), device=DEV)                    # unwritten while its pieces wait
    ws.pending = PendingUpdate(y, Partials(dev32(pieces), splits, T, D), accumulate=False)
    X = dev32(x)
    h = ops.rms_join(X, y, dev32(post), 1e-4, dev32(nxt), 1e-5, torch.float32, ws=ws)
    assert ws.pending is None and ws.counts["added_by_join"] == 1
    close(X, new, "stream")
    close(h, P.rms_norm(new, nxt, 1e-5), "h")


@pytest.mark.parametrize("T,D,E,top", [(9, 128, 5, 2), (3, 90, 4, 4), (40, 256, 9, 6), (5, 64, 1, 1)])
def test_joining_sums_a_token_s_experts(T, D, E, top):
    from photon_infer_amd import ops
    g = torch.Generator().manual_seed(3)
    ids = torch.stack([torch.randperm(E, generator=g)[:top] for _ in range(T)]).to(torch.int32)
    rows = ops.group_entries(ids.to(DEV), E)
    x, Y, w, post, nxt = randn(T, D, seed=1), randn(T * top, D, seed=2), torch.rand(T, top, generator=g, dtype=F64), randn(D, seed=3), randn(D, seed=4)
    where = rows.entry_row.cpu().long().view(T, top)
    y = (w.unsqueeze(2) * Y[where]).sum(1)
    new = x + P.rms_norm(y, post, 1e-4)
    X, hole = dev32(x), torch.full((T, D), float("nan"), device=DEV)
    h = ops.rms_join(X, hole, dev32(post), 1e-4, dev32(nxt), 1e-5, torch.float32, choices=ops.LeftChoices(hole, dev32(Y), dev32(w), rows))
    close(X, new, "stream")
    close(h, P.rms_norm(new, nxt, 1e-5), "h")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("sizes", [(6, 2, 48, 3, 2), (9, 2, 64, 3, 1), (7, 1, 36, 1, 1), (4, 4, 128, 1, 1), (1, 1, 48, 1, 1), (8, 3, 32, 4, 1 + 1), (4, 2, 20, 4, 2)])
@pytest.mark.parametrize("T", [1, 9, 150])
def test_routed_feed_forward_in_groups(dtype, sizes, T):
    from photon_infer_amd.parts import FEED_FORWARDS
    E, top, F, count, keep = sizes
    D, tdt = 64, TORCH[dtype]
    rnd = lambda *s, seed, scale=0.2: randn(*s, seed=seed, scale=scale).to(torch.bfloat16).double()
    W = {"router": rnd(E, D, seed=1, scale=0.3)}
    for e in range(E):
        W[f"e{e}.gate"], W[f"e{e}.up"], W[f"e{e}.down"] = rnd(F, D, seed=10 + e), rnd(F, D, seed=30 + e), rnd(D, F, seed=50 + e)
    part = FEED_FORWARDS.make("routed_experts", hidden_size=D, expert_size=F, num_experts=E, top=top, groups=count, keep=keep, accumulate=False)
    part.load({n: t.to(tdt).to(DEV) for n, t in W.items()}, tdt, torch.device(DEV))
    h = randn(T, D, seed=3).to(tdt).double()
    mlp = {"router": {"experts": E, "top": top, "groups": {"count": count, "keep": keep}}}
    with RouteRecorder() as rec:
        out = torch.full((T, D), 7.0, device=DEV)
        part.forward(h.to(tdt).to(DEV), out, SimpleNamespace(workspace=None, may_defer=False))
    ids, margins, chosen = rec.calls[0], [], []
    want = P.routed_ff(h, mlp, W, P.bf16_round if dtype == "bfloat16" else None, experts=ids.tolist(), margins=margins, chosen=chosen)
    for t in range(T):
        assert sorted(ids[t].tolist()) == sorted(chosen[t]) or (dtype == "bfloat16" and margins[t] < 0.02), (t, ids[t].tolist(), chosen[t], margins[t])
    close(out, want, f"{sizes} {T} tokens", 3e-5 if dtype == "float32" else 2e-2)


def test_squared_relu_and_factor_on_the_logits():
    from photon_infer_amd.parts import FEED_FORWARDS, RMSNorm
    D, F, T = 40, 56, 7
    for tdt in (torch.float32, torch.bfloat16):
        W = {"up": randn(F, D, seed=1, scale=0.3).to(torch.bfloat16).double(), "down": randn(D, F, seed=2, scale=0.3).to(torch.bfloat16).double()}
        part = FEED_FORWARDS.make("squared_relu_mlp", hidden_size=D, intermediate_size=F, accumulate=False)
        part.load({n: t.to(tdt).to(DEV) for n, t in W.items()}, tdt, torch.device(DEV))
        h, out = randn(T, D, seed=3).to(tdt).double(), torch.full((T, D), 9.0, device=DEV)
        part.forward(h.to(tdt).to(DEV), out, SimpleNamespace(workspace=None, may_defer=False))
        close(out, P.dense_ff(h, W, P.bf16_round if tdt == torch.bfloat16 else None), "squared relu", 3e-5 if tdt == torch.float32 else 1e-2)
        norm = RMSNorm(D, 1e-3, tensor_name="", mult=-1.75)
        w = torch.rand(D, dtype=F64) + 0.5
        norm.load({"": w.to(torch.bfloat16).to(DEV)}, tdt, torch.device(DEV))
        x = randn(T, D, seed=5)
        close(norm.forward(dev32(x)), -1.75 * P.rms_norm(x, w.to(torch.bfloat16).double(), 1e-3), "norm with a factor", act_tol("float32" if tdt == torch.float32 else "bfloat16"))


# ----------------------------------------------------------------------------- whole models
@pytest.fixture(scope="module")
def model_dirs(tmp_path_factory):
    root = tmp_path_factory.mktemp("roserax")
    return {name: TR.make_model_dir(root, name, seed=5) for name in TR.ALL}


_plain = {}
CLOSE_CALL = 0.05      # a bfloat16 choice that differs from the plain one must be this close to a tie (in the scores' logarithms)


def plain_logits(model_dir, tokens, emulate=False):
    key = (model_dir, tuple(tokens), emulate)
    if key not in _plain:
        cfg, W = P.read_model_folder(model_dir)
        _plain[key] = P.forward(cfg, W, list(tokens), P.bf16_round if emulate else None).float()
    return _plain[key]


def runner_for(model_dir, name, dtype, max_tokens):
    from photon_infer_amd.engine.replay import make_runner
    return make_runner(model_dir, dtype, max(max_tokens, 64), TR.ALL[name][1]["block_size"])


def check(got, model_dir, reqs, dtype, what, choices=None):
    """``choices`` (bfloat16 runs): the experts the engine chose per request; the plain logits are then those of the same choices,
    which must be the plain ones up to close calls."""
    assert got, "no logits came back"
    for rid, toks in reqs.items():
        forced = choices.get(rid) if choices else None
        if forced:
            cfg, W = P.read_model_folder(model_dir)
            margins, chosen, exact = {}, {}, {}
            emulated = P.forward(cfg, W, list(toks), P.bf16_round, experts=forced, margins=margins, chosen=chosen).float()
            ref = P.forward(cfg, W, list(toks), experts=forced, margins=exact).float()
            for i, ids in forced.items():
                # a close call: within three times of what the rounding moves this layer's margins by
                close_call = max(CLOSE_CALL, 3.0 * max((abs(a - b) for a, b in zip(margins[i], exact[i]) if math.isfinite(a)), default=0.0))
                for t in range(len(toks)):
                    if sorted(ids[t]) != sorted(chosen[i][t]):
                        assert margins[i][t] < close_call, f"{what}: layer {i} token {t}: experts {ids[t]} instead of {chosen[i][t]} (margin {margins[i][t]:.4f})"
        else:
            ref = plain_logits(model_dir, toks)
        if dtype == "float32":
            tol = 1e-4 * max(1.0, float(ref.abs().max()))
        else:       # three times what rounding activations to bfloat16 does to the plain implementation itself
            tol = 3.0 * float(((emulated if forced else plain_logits(model_dir, toks, True)) - ref).abs().max())
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


LENGTHS = {"A": [1, 26, 110], "B": [3, 70, 160], "C": [2, 30, 75], "D": [2, 45, 90], "E": [1, 66, 140]}


def requests_for(name, seed=0):
    vocab = TR.ALL[name][0]["vocab"]
    return {f"r{i}": random_tokens(n, vocab, seed * 100 + i) for i, n in enumerate(LENGTHS[name])}


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(TR.ALL))
def test_whole_prompts_and_the_stream_after_every_layer(name, dtype, model_dirs, tmp_path):
    reqs = requests_for(name)
    steps = []
    for rid, toks in reqs.items():
        steps += cut_steps(rid, toks, [len(toks)], first_step=len(steps))
    runner = runner_for(model_dirs[name], name, dtype, live_token_need(steps))
    run_checked(runner, steps, str(tmp_path), model_dirs[name], reqs, dtype, "whole")
    if dtype == "float32":         # a layer's last result is left to the next reader: it is applied to a copy here
        from photon_infer_amd.engine.step import StepEntry
        from photon_infer_amd.parts.norm import LEFT_JOIN
        toks = reqs["r2"]
        cfg, W = P.read_model_folder(model_dirs[name])
        want, got = [], []
        P.forward(cfg, W, toks, streams=want)
        for blk in runner.model.blocks:
            def wrapped(x, ctx, cache, f=blk.forward):
                f(x, ctx, cache)
                left = ctx.scratch[LEFT_JOIN]
                assert left.x is x
                kept = x.clone()
                y = left.y if left.choices is None else torch.empty_like(x)
                if left.choices is not None:
                    from photon_infer_amd import ops
                    ops.combine_choices(y, left.choices.y, left.choices.weights, left.choices.rows)
                else:
                    from photon_infer_amd import ops
                    ops.materialize(y, ctx.workspace)
                got.append(kept.double().cpu() + P.rms_norm(y.double().cpu(), left.weight.double().cpu(), left.eps))
            blk.forward = wrapped
        runner.admit("s")
        runner.step([StepEntry("s", toks, [])])
        assert len(got) == len(want) == len(cfg["layers"])
        for i, (g, w) in enumerate(zip(got, want)):
            close(g, w, f"stream after layer {i}", 1e-4)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(TR.ALL))
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
@pytest.mark.parametrize("name", list(TR.ALL))
@pytest.mark.parametrize("sizes", [[2], [7, 2, 31, 1, 3], [64, 5], [17]])
def test_portions_of_changing_size(name, dtype, sizes, model_dirs, tmp_path):
    reqs = {"r2": requests_for(name, seed=2)["r2"]}
    steps = cut_steps("r2", reqs["r2"], sizes)
    runner = runner_for(model_dirs[name], name, dtype, live_token_need(steps))
    run_checked(runner, steps, str(tmp_path), model_dirs[name], reqs, dtype, f"portions {sizes}")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(TR.ALL))
def test_mixed_batches_with_pages_and_slots_used_again(name, dtype, model_dirs, tmp_path):
    """Seven unequal requests through four slots: some bring portions while others decode, and now and then single tokens
    only; a request may sit out a step; a finished request's pages and slot go to the next one.  Each must come out as it does alone."""
    vocab = TR.ALL[name][0]["vocab"]
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
    runner.cache.check_invariants()


@pytest.mark.parametrize("dtype", DTYPES)
def test_a_long_prompt_whole_and_in_two_long_portions(dtype, model_dirs, tmp_path):
    vocab = TR.ALL["A"][0]["vocab"]
    reqs = {"w": random_tokens(420, vocab, 11), "p": random_tokens(420, vocab, 11)}
    steps = cut_steps("w", reqs["w"], [420])
    steps += cut_steps("p", reqs["p"], [201, 218, 1], first_step=len(steps))
    runner = runner_for(model_dirs["A"], "A", dtype, live_token_need(steps))
    run_checked(runner, steps, str(tmp_path), model_dirs["A"], reqs, dtype, "long prompt")


@pytest.mark.parametrize("name", ["A", "B", "C", "D"])
def test_long_decoding_keeps_state_and_first_tokens_and_gives_pages_back(name, model_dirs, tmp_path):
    """250 tokens one by one after a portion of three over a pool of 256: windows pass over decoded tokens and hand their pages back,
    the kept tokens' pages stay."""
    vocab = TR.ALL[name][0]["vocab"]
    toks = random_tokens(250, vocab, 9)
    steps = cut_steps("long", toks, [3] + [1] * 247, end=False)
    runner = runner_for(model_dirs[name], name, "float32", 256)
    run_checked(runner, steps, str(tmp_path), model_dirs[name], {"long": toks}, "float32", "long decoding")
    page, ceil = TR.ALL[name][1]["block_size"], lambda a, b: -(-a // b)
    for g in runner.cache.groups:
        first = max(0, 250 - g.window + 1) // page if g.window is not None else 0
        kept = ceil(g.keep_first, page) if g.window is not None else 0
        assert g.pool.num_allocated == ceil(250, page) - first + min(kept, first), (g.window, g.keep_first)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(TR.ALL))
def test_greedy_generation_through_the_engine(name, dtype, model_dirs):
    """The engine's own entry point, scheduler, sampling and decode steps: unequal prompts at once, more requests than slots,
    prompts longer than a portion; every request must generate what the plain implementation generates alone."""
    from photon_infer_amd.engine import ContinuousBatchEngine, EngineOptions
    cfg, W = P.read_model_folder(model_dirs[name])
    vocab = cfg["vocab"]
    prompts = [random_tokens(n, vocab, 70 + i) for i, n in enumerate([5, 41, 18, 70, 2])]
    engine = ContinuousBatchEngine(model_dirs[name], EngineOptions(dtype=dtype, block_size=TR.ALL[name][1]["block_size"], max_batch=3,
                                                                   max_cache_tokens=1024, chunk_size=32, max_model_len=200))
    got = engine.generate(prompts, max_new_tokens=10)
    for prompt, out in zip(prompts, got):
        want = P.greedy(cfg, W, prompt, 10)
        if dtype == "float32":
            assert list(out) == want
        else:       # bfloat16: a near tie may fall the other way; the differing token must be a close second of the
            # plain logits
            for i, (a, b) in enumerate(zip(out, want)):
                if a != b:
                    margins = {}
                    lg = P.forward(cfg, W, prompt + want[:i], margins=margins)[-1]
                    if min((m for v in margins.values() for m in v), default=1.0) < CLOSE_CALL:
                        break                          # a routing choice on the way was a close call: another expert, another token
                    tol = 3.0 * float((P.forward(cfg, W, prompt + want[:i], P.bf16_round)[-1] - lg).abs().max())
                    assert float(lg[b] - lg[a]) <= 2.0 * tol, f"token {i}: {a} instead of {b} ({float(lg[b] - lg[a]):.3f} apart, bound {tol:.3f})"
                    break


def test_command_line_and_replayed_decode_steps(model_dirs, tmp_path):
    """The framework's commands serve the design as they serve its others (from a folder, and from a bare configuration with
    random weights); and decode steps replayed as HIP graphs give the tokens of eager steps, with new requests' prompts in
    between and states and pages that are used again."""
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
    assert "Architecture: Roserax" in proc.stdout and f"Generated ids: {','.join(map(str, want))}" in proc.stdout
    (tmp_path / "cfg").mkdir()
    json.dump(TR.TINY_E, open(tmp_path / "cfg" / "config.json", "w"))
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

    for name in ("A", "B"):
        vocab = TR.ALL[name][0]["vocab"]
        prompts = [random_tokens(n, vocab, 90 + n) for n in (3, 40, 17, 9, 26)]

        def run(use_graphs):
            eng = ContinuousBatchEngine(model_dirs[name], EngineOptions(dtype="bfloat16", block_size=16, max_batch=3, max_cache_tokens=1024,
                                                                        chunk_size=8, max_step_tokens=24, max_model_len=200, use_graphs=use_graphs))
            assert eng.runner.graph_safe
            out = eng.generate(prompts, max_new_tokens=40, ignore_eos=True)
            return out, eng.runner.graphs_captured

        graphs, captured = run(True)
        eager, none = run(False)
        assert captured > 0 and none == 0
        assert [list(o) for o in graphs] == [list(o) for o in eager]


def wide_config():
    attn = TR._attn(16, 4, 64, 64, 0.12, 150, 20)
    lat = TR._latent(8, 64, 32, 128, 384, 160, 0.1, 10000.0)
    ret = TR._ret(128, 64, [1.0 - 2.0 ** -(3 + i) for i in range(8)], 10000.0, 128)
    moe = TR._moe(512, 8, 3, 4, 2)
    return TR._model(1000, 1024, 4.0, 0.5, 1e-5, [TR._layer("attention", attn, TR._dense(3072)), TR._layer("latent_attention", lat, moe),
                                                  TR._layer("retention", ret, moe), TR._layer("attention", attn, TR._dense(2048))])


def test_kernels_chosen_at_real_widths_against_the_general_kernels(tmp_path):
    """A model wide enough that the bfloat16 engine takes what it takes at real sizes (tile products with their epilogues for the
    prompt, weight-streaming products left in pieces for single tokens, the matrix-core attention, grouped tile products) against
    the same engine on the general kernels: a 300-token prompt, a mixed step and decode steps of a batch, the same experts in both."""
    from photon_infer_amd import ops
    from photon_infer_amd.config import RoseraxConfig
    from photon_infer_amd.engine.replay import make_runner
    from photon_infer_amd.engine.step import StepEntry
    from photon_infer_amd.weights import write_random_model
    d = write_random_model(RoseraxConfig.from_dict(wide_config()), str(tmp_path / "wide"), seed=2, std=0.03, norm_init="uniform", dtype="bfloat16")
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
            return forced, torch.softmax(a[0], dim=-1).gather(1, forced.long()).contiguous()
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
                assert r.workspace.counts["added_by_join"] > 0
        finally:
            ops.route = real
            ops.use_fast_kernels(prev)
    err = float((outs[0] - outs[1]).abs().max())
    assert err <= 0.04 * float(outs[1].std()) + 0.02, (err, float(outs[1].std()))
