"""Plain implementation of the Roserax design: whole sequences, no cache, float64, one function per mechanism.  It shares
nothing with the engine: it takes the raw config.json mapping and a dict of tensors by their names in a model folder.

    x = embed[token] * scale
    per layer:  x <- x + rms(mixer(rms(x; norm1)); norm1b);  x <- x + rms(ff(rms(x; norm2)); norm2b)   (layers with a feed-forward)
    logits = logit_scale * embed . rms(x; final.norm)

A layer's mixer is attention within a window that keeps a sequence's first tokens (no positions in the scores, a one in the
softmax's denominator), attention through a latent with a gate per feature, or retention (a matrix state per head with a
fixed decay).
"""
from __future__ import annotations

import json
import math
import os
from typing import Callable, Dict, List, Optional

import torch

F64 = torch.float64
Round = Optional[Callable[[torch.Tensor], torch.Tensor]]


def bf16_round(t: torch.Tensor) -> torch.Tensor:
    return t.to(torch.bfloat16).to(t.dtype)


def _r(t: torch.Tensor, act_round: Round) -> torch.Tensor:
    """Activations rounded where an engine that computes in a 16-bit type rounds them (None: not at all)."""
    return act_round(t.to(torch.float32)).to(F64) if act_round is not None else t


def read_model_folder(model_dir: str):
    """(raw config.json, tensors by name) of a model folder written with safetensors."""
    from safetensors.torch import load_file
    with open(os.path.join(model_dir, "config.json"), encoding="utf-8") as f:
        config = json.load(f)
    return config, load_file(os.path.join(model_dir, "model.safetensors"))


def rms_norm(x: torch.Tensor, w: Optional[torch.Tensor], eps: float) -> torch.Tensor:
    """x / sqrt(mean(x^2) + eps) [* w] over the last axis."""
    y = x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)
    return y if w is None else y * w


def sigmoid(x: torch.Tensor) -> torch.Tensor:
    return 1.0 / (1.0 + torch.exp(-x))


def silu(x: torch.Tensor) -> torch.Tensor:
    return x * sigmoid(x)


def kept_window_mask(T: int, size: Optional[int], keep_first: int) -> torch.Tensor:
    """[T, T] bool: query i sees key j when j <= i and the key is one of the last ``size`` up to i or one of the first ``keep_first``."""
    seen = torch.zeros((T, T), dtype=torch.bool)
    for i in range(T):
        for j in range(i + 1):
            seen[i, j] = size is None or i - j < size or j < keep_first
    return seen


def causal_mask(T: int) -> torch.Tensor:
    return kept_window_mask(T, None, 0)


def softmax_over(s: torch.Tensor, seen: torch.Tensor, one: bool) -> torch.Tensor:
    """Rows of weights exp(s) / (sum over the seen keys of exp(s), plus 1 with ``one``); unseen keys weigh nothing."""
    s = torch.where(seen, s, torch.full_like(s, -math.inf))
    m = s.max(dim=-1, keepdim=True).values
    if one:
        m = torch.clamp(m, min=0.0)
    e = torch.exp(s - m)
    den = e.sum(dim=-1, keepdim=True)
    return e / (den + torch.exp(-m) if one else den)


def rotate_halves(x: torch.Tensor, positions: torch.Tensor, dims: int, base: float) -> torch.Tensor:
    """x [T, ..., d]: of the first ``dims`` features, i and i + dims / 2 turned by position * base^(-2 i / dims); the rest as they are."""
    y = x.clone()
    half = dims // 2
    shape = [x.shape[0]] + [1] * (x.dim() - 2)
    for i in range(half):
        a = positions.to(F64) * base ** (-2.0 * i / dims)
        c, s = torch.cos(a).reshape(shape), torch.sin(a).reshape(shape)
        u, v = x[..., i], x[..., i + half]
        y[..., i] = u * c - v * s
        y[..., i + half] = v * c + u * s
    return y


def window_attention(h: torch.Tensor, m: dict, W: Dict[str, torch.Tensor], eps: float, act_round: Round = None) -> torch.Tensor:
    T, H, G, d, dv = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = _r(rms_norm((h @ W["q"].T).reshape(T, H, d), W["q.norm"], eps), act_round)
    k = _r(rms_norm((h @ W["k"].T).reshape(T, G, d), W["k.norm"], eps), act_round)
    v = _r((h @ W["v"].T).reshape(T, G, dv), act_round)
    mask = m.get("mask") or {}
    seen = kept_window_mask(T, mask.get("size"), mask.get("keep_first", 0))
    out = torch.zeros((T, H, dv), dtype=F64)
    for n in range(H):
        g = n // (H // G)
        p = softmax_over((q[:, n] @ k[:, g].T) * m["scale"], seen, one=True)
        out[:, n] = p @ v[:, g]
    return _r(out.reshape(T, H * dv), act_round) @ W["o"].T


def latent_attention(h: torch.Tensor, m: dict, W: Dict[str, torch.Tensor], eps: float, act_round: Round = None) -> torch.Tensor:
    """Keys and values written out per head, as the definition has them."""
    T, H, d, dr, dv, rank = h.shape[0], m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    positions = torch.arange(T)
    turn = lambda t: rotate_halves(t, positions, m["rot"]["dims"], float(m["rot"]["base"])) if dr else t
    cq = _r(rms_norm(h @ W["dq"].T, W["dq.norm"], eps), act_round)
    q = _r(cq @ W["uq"].T, act_round).reshape(T, H, d + dr)
    q_rot = turn(q[..., d:])
    down = h @ W["dkv"].T
    c = _r(rms_norm(down[:, :rank], W["dkv.norm"], eps), act_round)
    k_rot = _r(turn(down[:, rank:]), act_round)
    k_plain = (c @ W["uk"].T).reshape(T, H, d)
    v = (c @ W["uv"].T).reshape(T, H, dv)
    seen = causal_mask(T)
    out = torch.zeros((T, H, dv), dtype=F64)
    for n in range(H):
        s = (q[:, n, :d] @ k_plain[:, n].T + q_rot[:, n] @ k_rot.T) * m["scale"]
        out[:, n] = softmax_over(s, seen, one=False) @ v[:, n]
    return _r(out.reshape(T, H * dv) * sigmoid(h @ W["g"].T), act_round) @ W["o"].T


def retention_heads(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, decay: List[float], state: Optional[torch.Tensor] = None):
    """Token by token: S <- decay S + k v^T, o = S^T q per head.  q, k [T, H, d], v [T, H, dv]; ``state`` [H, d, dv] is what the
    sequence starts from (None: zero).  Returns (o [T, H, dv], the state behind the last token)."""
    T, H, d = q.shape
    S = torch.zeros((H, d, v.shape[2]), dtype=F64) if state is None else state.clone()
    g = torch.tensor(decay, dtype=F64).reshape(H, 1, 1)
    o = torch.zeros((T, H, v.shape[2]), dtype=F64)
    for t in range(T):
        S = g * S + k[t].unsqueeze(2) * v[t].unsqueeze(1)
        o[t] = (S * q[t].unsqueeze(2)).sum(dim=1)
    return o, S


def retention(h: torch.Tensor, m: dict, W: Dict[str, torch.Tensor], eps: float, act_round: Round = None) -> torch.Tensor:
    T, H, d, dv = h.shape[0], m["heads"], m["dim"], m["vdim"]
    positions = torch.arange(T)
    dims, base = m["rot"]["dims"], float(m["rot"]["base"])
    q = rotate_halves((h @ W["q"].T).reshape(T, H, d), positions, dims, base)
    k = rotate_halves((h @ W["k"].T).reshape(T, H, d), positions, dims, base) * d ** -0.5
    o, _ = retention_heads(q, k, (h @ W["v"].T).reshape(T, H, dv), m["decay"])
    o = rms_norm(o, None, eps).reshape(T, H * dv)
    return _r(o * silu(h @ W["g"].T), act_round) @ W["o"].T


def dense_ff(h: torch.Tensor, W: Dict[str, torch.Tensor], act_round: Round = None) -> torch.Tensor:
    u = torch.clamp(h @ W["up"].T, min=0.0)
    return _r(u * u, act_round) @ W["down"].T


def choose_experts(scores: torch.Tensor, top: int, groups: int, keep: int) -> List[int]:
    """The experts of one token: the ``keep`` groups of neighbours with the largest best score, then the ``top`` best in them."""
    E = scores.numel()
    per = E // groups
    best = sorted(range(groups), key=lambda g: (-float(scores[g * per:(g + 1) * per].max()), g))[:keep]
    allowed = [e for e in range(E) if e // per in best]
    return sorted(allowed, key=lambda e: (-float(scores[e]), e))[:top]


def choice_margin(scores: torch.Tensor, top: int, groups: int, keep: int) -> float:
    """How far the choice of one token is from another: the least distance, in the scores' logarithms, between something chosen
    and something passed over - groups among groups, experts within the chosen groups."""
    logs = torch.log(scores)
    best = torch.sort(logs.reshape(groups, -1).max(dim=1).values, descending=True).values
    within = torch.sort(logs[choose_experts(scores, keep * (scores.numel() // groups), groups, keep)], descending=True).values
    gaps = [float(best[keep - 1] - best[keep])] if keep < groups else []
    gaps += [float(within[top - 1] - within[top])] if top < within.numel() else []
    return min(gaps, default=math.inf)


def routed_ff(h: torch.Tensor, mlp: dict, W: Dict[str, torch.Tensor], act_round: Round = None, experts=None, margins: Optional[list] = None,
              chosen: Optional[list] = None) -> torch.Tensor:
    """``experts``: the choices to make instead of the router's own ([T][top] expert numbers); ``margins`` collects how far each
    token's own choice is from another (``choice_margin``), ``chosen`` the own choices."""
    r = mlp["router"]
    groups = r.get("groups") or {"count": 1, "keep": 1}
    scores = torch.softmax(h @ W["router"].T, dim=-1)
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        own = choose_experts(scores[t], r["top"], groups["count"], groups["keep"])
        if margins is not None:
            margins.append(choice_margin(scores[t], r["top"], groups["count"], groups["keep"]))
        if chosen is not None:
            chosen.append(own)
        for e in own if experts is None else experts[t]:
            act = _r(silu(h[t] @ W[f"e{e}.gate"].T) * (h[t] @ W[f"e{e}.up"].T), act_round)
            out[t] += scores[t, e] * (act @ W[f"e{e}.down"].T)
    return out


MIXERS = {"attention": window_attention, "latent_attention": latent_attention, "retention": retention}


def _sub(tensors: Dict[str, torch.Tensor], prefix: str) -> Dict[str, torch.Tensor]:
    return {n[len(prefix):]: t.to(F64) for n, t in tensors.items() if n.startswith(prefix)}


def forward(config: dict, tensors: Dict[str, torch.Tensor], tokens, act_round: Round = None, streams: Optional[list] = None,
            experts: Optional[dict] = None, margins: Optional[dict] = None, chosen: Optional[dict] = None) -> torch.Tensor:
    """float64 logits [T, vocab] of one whole sequence; ``streams`` collects the stream after every layer; ``experts``:
    {layer: [T][top]} choices to make instead of the routers' own; ``margins`` and ``chosen`` collect per layer what
    ``routed_ff`` collects."""
    eps = float(config["norm"]["eps"])
    embed = tensors["embed"].to(F64)
    norm = lambda x, name: rms_norm(x, tensors[name].to(F64), eps)
    x = embed[torch.as_tensor(list(tokens), dtype=torch.long)] * float(config["embedding"]["scale"])
    for i, layer in enumerate(config["layers"]):
        h = _r(norm(x, f"l{i}.norm1"), act_round)
        y = MIXERS[layer["type"]](h, layer["mixer"], _sub(tensors, f"l{i}.mix."), eps, act_round)
        x = x + norm(y, f"l{i}.norm1b")
        mlp = layer.get("mlp")
        if mlp is not None:
            h = _r(norm(x, f"l{i}.norm2"), act_round)
            W = _sub(tensors, f"l{i}.mlp.")
            if mlp["kind"] == "dense":
                y = dense_ff(h, W, act_round)
            else:
                keep = lambda d: d.setdefault(i, []) if d is not None else None
                y = routed_ff(h, mlp, W, act_round, (experts or {}).get(i), keep(margins), keep(chosen))
            x = x + norm(y, f"l{i}.norm2b")
        if streams is not None:
            streams.append(x.clone())
    return _r(norm(x, "final.norm"), act_round) @ embed.T * float(config["logit_scale"])


def greedy(config: dict, tensors: Dict[str, torch.Tensor], prompt, new_tokens: int) -> List[int]:
    """Greedy continuation, the whole sequence run again for every token."""
    seq = list(prompt)
    for _ in range(new_tokens):
        seq.append(int(torch.argmax(forward(config, tensors, seq)[-1])))
    return seq[len(prompt):]
