"""Helpers shared by the GPU tests."""
from __future__ import annotations

import io
import json
import os
from types import SimpleNamespace
from typing import Dict, List, Sequence

import numpy as np
import torch

DEV = "cuda:0"


def fp32_tol(ref: torch.Tensor) -> float:
    """float32 engine against the float32 plain implementation."""
    return 3e-5 * max(1.0, ref.abs().max().item())


def bf16_tol(ref: torch.Tensor, emulated: torch.Tensor) -> float:
    """bfloat16 engine against the float32 plain implementation.  The yardstick is what
    rounding activations to bfloat16 at the engine's rounding points does to the plain
    implementation itself (``emulated``): the engine may be off by three times the largest
    deviation that this rounding causes anywhere in the sequence, and no more."""
    return 3.0 * (emulated - ref).abs().max().item()


def tol_for(dtype: str, ref: torch.Tensor, emulated: torch.Tensor = None) -> float:
    return fp32_tol(ref) if dtype == "float32" else bf16_tol(ref, emulated)


class PagedKV:
    """Scatter dense per-request K/V [S, kv_heads, hd] into a page pool under a random page order."""

    def __init__(self, seqs: Sequence[tuple], page_size: int, dtype, seed: int = 0, spare_pages: int = 3):
        nkv, hd = seqs[0][0].shape[1:]
        vd = seqs[0][1].shape[2]          # values may have another width than keys
        blocks = [-(-k.shape[0] // page_size) for k, _ in seqs]
        total = sum(blocks) + spare_pages
        g = torch.Generator().manual_seed(seed)
        order = torch.randperm(total, generator=g).tolist()
        width = max(blocks)
        self.table = torch.full((len(seqs), width), -1, dtype=torch.int32)
        # unused pages hold large values: a read outside a request's keys shows
        self.k = torch.full((total, nkv, page_size, hd), 1e4, dtype=torch.float32)
        self.v = torch.full((total, nkv, vd, page_size), -1e4, dtype=torch.float32)   # values are kept transposed
        it = iter(order)
        for r, (k, v) in enumerate(seqs):
            for b in range(blocks[r]):
                page = next(it)
                self.table[r, b] = page
                n = min(page_size, k.shape[0] - b * page_size)
                self.k[page, :, :n] = k[b * page_size: b * page_size + n].transpose(0, 1)
                self.v[page, :, :, :n] = v[b * page_size: b * page_size + n].permute(1, 2, 0)
        self.k = self.k.to(dtype).to(DEV)
        self.v = self.v.to(dtype).to(DEV)
        self.table = self.table.to(DEV)
        self.page_size = page_size


def attention_ctx(q_lens: Sequence[int], kv_lens: Sequence[int], dtype) -> SimpleNamespace:
    """The fields of a StepContext that the attention kernels read, made as the step function makes them."""
    from photon_infer_amd import ops

    R = len(q_lens)
    q_start = np.zeros(R + 1, np.int32)
    np.cumsum(q_lens, out=q_start[1:])
    parts = {
        "positions": np.concatenate([np.arange(kv - n, kv, dtype=np.int32) for n, kv in zip(q_lens, kv_lens)]),
        "req_of_token": np.repeat(np.arange(R, dtype=np.int32), q_lens),
        "q_start": q_start, "kv_len": np.asarray(kv_lens, np.int32),
    }
    views = ops.upload_arrays(parts, DEV)
    # no runner here: no workspace (the ops take what they need per call) and no plans made
    # beforehand (the attention op makes its work list itself)
    return SimpleNamespace(T=int(sum(q_lens)), R=R, dtype=dtype, q_lens=list(q_lens), kv_lens=list(kv_lens),
                           max_q_len=max(q_lens), max_kv_len=max(kv_lens), all_decode=all(n == 1 for n in q_lens), scratch={},
                           workspace=None, plans={}, **{k: views[k] for k in ("positions", "req_of_token", "q_start", "kv_len")})


def run_trace(runner, steps: List[dict], out_dir: str) -> Dict[tuple, torch.Tensor]:
    """Replay ``steps`` through the framework's replay loop; {(id, position): logits row}."""
    from photon_infer_amd.engine.replay import replay

    lines = io.StringIO("\n".join(json.dumps(s) for s in steps) + "\n")
    done = io.StringIO()
    replay(runner, lines, out_dir, done)
    assert done.getvalue().split() == [w for s in steps for w in ("done", str(s["step"]))]
    return collect_logits(steps, out_dir, runner.spec.vocab_size)


def collect_logits(steps: List[dict], out_dir: str, vocab: int) -> Dict[tuple, torch.Tensor]:
    got, pos = {}, {}
    for s in steps:
        wanted = [(e["id"], pos.get(e["id"], 0) + w) for e in s["entries"] for w in e.get("want", [])]
        for e in s["entries"]:
            pos[e["id"]] = pos.get(e["id"], 0) + len(e["tokens"])
        for rid in s.get("end", []):
            pos.pop(rid, None)
        path = os.path.join(out_dir, f"{s['step']}.f32")
        if not wanted:
            assert not os.path.exists(path)
            continue
        arr = np.fromfile(path, dtype="<f4").reshape(len(wanted), vocab)
        for key, row in zip(wanted, arr):
            assert key not in got
            got[key] = torch.from_numpy(row.copy())
    return got


def cut_steps(rid: str, tokens: Sequence[int], sizes: Sequence[int], first_step: int = 0, want_all: bool = True,
              end: bool = True) -> List[dict]:
    """Steps that feed ``tokens`` of one request in portions of ``sizes`` (cycled)."""
    steps, i, k = [], 0, 0
    while i < len(tokens):
        n = min(sizes[k % len(sizes)], len(tokens) - i)
        steps.append({"step": first_step + len(steps),
                      "entries": [{"id": rid, "tokens": list(tokens[i:i + n]), "want": list(range(n)) if want_all else []}],
                      "end": []})
        i += n
        k += 1
    if end:
        steps[-1]["end"] = [rid]
    return steps


def live_token_need(steps: List[dict], rounding: int = 64) -> int:
    """The --max-tokens a trace needs: most tokens live at once, each request rounded up."""
    held, worst = {}, 0
    for s in steps:
        for e in s["entries"]:
            held[e["id"]] = held.get(e["id"], 0) + len(e["tokens"])
        worst = max(worst, sum(-(-n // rounding) * rounding for n in held.values()))
        for rid in s.get("end", []):
            held.pop(rid, None)
    return worst


# ------------------------------------------------------------------ inputs, comparisons and contexts for kernels on their own
def randn(*shape, seed=0, scale=1.0):
    return torch.randn(*shape, generator=torch.Generator().manual_seed(seed), dtype=torch.float64) * scale


def close(got, ref, what, tol=2e-5):
    tol = tol * max(1.0, float(ref.abs().max()))
    err = float((got.double().cpu() - ref).abs().max())
    assert err <= tol, f"{what}: error {err:.3e} > {tol:.3e}"


def dev32(t):
    return t.float().to(DEV).contiguous()


def state_ctx(q_lens, slots):
    """The fields of a StepContext that the kernels of mixers with a state read."""
    q_start = np.zeros(len(q_lens) + 1, np.int32)
    np.cumsum(q_lens, out=q_start[1:])
    return SimpleNamespace(T=int(sum(q_lens)), R=len(q_lens), max_q_len=max(q_lens), q_lens=list(q_lens),
                           q_start=torch.from_numpy(q_start).to(DEV), slots=torch.tensor(slots, dtype=torch.int32, device=DEV))


def in_steps(seqs, cuts):
    """Steps over several sequences at once: ``cuts[name]`` are the portion sizes of sequence ``name`` (cycled); a step
    holds the next portion of every sequence that has tokens left.  Yields [(name, begin, end)]."""
    at = {n: 0 for n in seqs}
    k = 0
    while any(at[n] < seqs[n] for n in seqs):
        step = []
        for n in seqs:
            if at[n] < seqs[n]:
                size = min(cuts[n][k % len(cuts[n])], seqs[n] - at[n])
                step.append((n, at[n], at[n] + size))
                at[n] += size
        k += 1
        yield step


def paged(lengths, page, seed=0):
    """(block table [requests, width] on the device, pages in the pool): pages dealt out of order, three to spare."""
    blocks = [-(-n // page) for n in lengths]
    total = sum(blocks) + 3
    order = torch.randperm(total, generator=torch.Generator().manual_seed(seed)).tolist()
    table = torch.full((len(lengths), max(blocks)), -1, dtype=torch.int32)
    it = iter(order)
    for r, b in enumerate(blocks):
        for j in range(b):
            table[r, j] = next(it)
    return table.to(DEV), total


def make_part(kind, tensors, tdt, **params):
    from photon_infer_amd.parts import MIXERS
    part = MIXERS.make(kind, **params)
    names = {s.name: s for s in part.tensor_specs()}
    assert set(names) == set(tensors), (sorted(names), sorted(tensors))
    part.load({n: t.to(tdt if t.dim() == 2 else torch.float32).to(DEV) for n, t in tensors.items()}, tdt, torch.device(DEV))
    return part


def run_paged_part(part, h, want, cuts_list, tdt, page, tol, what, D):
    """A mixer with pages as a part, on pages dealt out of order: under each cutting of the sequence its result must be the plain one."""
    from photon_infer_amd.parts import LayerCache
    T = h.shape[0]
    table, pages = paged([T], page, seed=2)
    spec = part.cache_spec()
    pools = {t.name: torch.zeros((pages, *t.page_shape(page)), dtype=tdt, device=DEV) for t in spec.tensors}
    cache = LayerCache(group=0, k=pools["k"], v=pools["v"], page_size=page, writes=True, tensors=pools)
    for cuts in cuts_list:
        for t in pools.values():
            t.fill_(50.0)                     # what a page held before must not show
        done = 0
        for n in cuts:
            ctx = attention_ctx([n], [done + n], tdt)
            ctx.block_tables, ctx.may_defer = {0: table}, False
            x = torch.full((n, D), 3.0, dtype=torch.float32, device=DEV)          # the part writes its result, it does not add
            part.forward(h[done:done + n].to(tdt).to(DEV).contiguous(), x, ctx, cache)
            close(x, want[done:done + n], f"{what} tokens {done} .. {done + n} of cuts {cuts[:4]}", tol)
            done += n


class RouteRecorder:
    """Records the experts the engine chooses (every call of ``ops.route``, in order), so that the plain implementation can be
    asked for the logits of the same choices: among hundreds of routing decisions some are near ties, which bfloat16 rounding
    decides either way, and one flipped expert changes everything after it."""

    def __enter__(self):
        from photon_infer_amd import ops
        self.ops, self.real, self.calls = ops, ops.route, []

        def route(*a, **k):
            ids, w = self.real(*a, **k)
            self.calls.append(ids.cpu())
            return ids, w
        ops.route = route
        return self

    def __exit__(self, *exc):
        self.ops.route = self.real

    def by_request(self, steps, config):
        """{request: {routed layer: [tokens, top] expert ids}} from the calls, given the trace's steps."""
        layers = [i for i, l in enumerate(config["layers"]) if l["mlp"] and l["mlp"]["kind"] == "moe"]
        out, k = {}, 0
        for s in steps:
            sizes = [len(e["tokens"]) for e in s["entries"]]
            for i in layers:
                for e, part in zip(s["entries"], torch.split(self.calls[k], sizes)):
                    out.setdefault(e["id"], {}).setdefault(i, []).append(part)
                k += 1
        assert k == len(self.calls)
        return {rid: {i: [r.tolist() for r in torch.cat(p)] for i, p in per.items()} for rid, per in out.items()}
