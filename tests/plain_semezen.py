"""Plain implementation of the Semezen design: whole sequences, no cache, float64, loops over
positions and heads, one function per mechanism.  It shares nothing with the engine: it takes
the raw config.json mapping and a dict of tensors by their names in a model folder.

    X_s = embed[token]                                          (s = 1 .. streams copies)
    per layer and sublayer (1: the mixer, 2: the feed-forward, where there is one):
        u = sum_s in_s X_s;   y = sublayer(rms(u; norm));   X_t <- sum_s mix[s, t] X_s + out_t y
    logits = head . rms(sum_s X_s; final.norm)

What a mixer reads is h + (h' - h) * shift, with h the normalised u of the token and h' that of its left
neighbour (the first token's is zero).  A layer's mixer is one of

* ``attention``: grouped-query attention within a sliding window; queries and keys with biases,
  a part of each head rotated (paired halves, frequencies scaled by wavelength), then every head
  of both divided by its root mean square; value vectors are the biased keys, unturned and at their own length; every
  feature of the result times a sigmoid gate;
* ``mingru``: ``S <- (1 - z) S + z c`` per feature with ``z = sigmoid(Wz h + bz)``, ``u = Wx h + bx``,
  ``c = u + 1/2`` for u >= 0 and ``sigmoid(u)`` below; the result is ``Wo (S * silu(Wg h))``.

A feed-forward is ``W_down gelu(W_up h)``, or routed: sigmoid scores, the largest ``top`` of them, each
chosen expert a clamped gated unit fed with ``score * h``, the results added.
"""
from __future__ import annotations

import json
import math
import os
from typing import Callable, Dict, List, Optional

import torch

F64 = torch.float64
Round = Optional[Callable[[torch.Tensor], torch.Tensor]]
GLU_ALPHA = 1.702


def bf16_round(t: torch.Tensor) -> torch.Tensor:
    return t.to(torch.bfloat16).to(t.dtype)


def _r(t: torch.Tensor, act_round: Round) -> torch.Tensor:
    """Activations rounded where an engine that computes in a 16-bit type rounds them (None: not at all)."""
    return act_round(t.to(torch.float32)).to(F64) if act_round is not None else t


def read_model_folder(model_dir: str):
    from safetensors.torch import load_file
    with open(os.path.join(model_dir, "config.json"), encoding="utf-8") as f:
        config = json.load(f)
    return config, load_file(os.path.join(model_dir, "model.safetensors"))


# ------------------------------------------------------------------ small functions
def rms_norm(x: torch.Tensor, w: Optional[torch.Tensor], eps: float) -> torch.Tensor:
    y = x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)
    return y if w is None else y * w


def sigmoid(x: torch.Tensor) -> torch.Tensor:
    return 1.0 / (1.0 + torch.exp(-x))


def silu(x: torch.Tensor) -> torch.Tensor:
    return x * sigmoid(x)


def gelu(x: torch.Tensor) -> torch.Tensor:
    """x Phi(x), Phi the normal distribution function."""
    return 0.5 * x * (1.0 + torch.erf(x / math.sqrt(2.0)))


def shift_in(h: torch.Tensor, share: torch.Tensor) -> torch.Tensor:
    """h [T, D]: every token moved towards the token before it by ``share`` (zeros stand before the first)."""
    out = h.clone()
    for t in range(h.shape[0]):
        before = h[t - 1] if t else torch.zeros_like(h[0])
        out[t] = h[t] + (before - h[t]) * share
    return out


def mix_streams(X: List[torch.Tensor], y: torch.Tensor, mix: torch.Tensor, out: torch.Tensor) -> List[torch.Tensor]:
    """Every new stream from the streams as they were: X_t <- sum_s mix[s, t] X_s + out[t] y."""
    n = len(X)
    return [sum(mix[s, t] * X[s] for s in range(n)) + out[t] * y for t in range(n)]


def rope_frequency(i: int, dims: int, base: float, scaling: Optional[dict]) -> float:
    """The i-th pair's angle per position: short waves as they are, long ones slowed by the factor, those between blended."""
    f = base ** (-2.0 * i / dims)
    if not scaling:
        return f
    wave, L = 2.0 * math.pi / f, float(scaling["original"])
    lo, hi, factor = float(scaling["low"]), float(scaling["high"]), float(scaling["factor"])
    if wave < L / hi:
        return f
    if wave > L / lo:
        return f / factor
    s = (L / wave - lo) / (hi - lo)
    return (1.0 - s) * f / factor + s * f


def rotate_halves(x: torch.Tensor, pos: int, dims: int, base: float, scaling: Optional[dict] = None) -> torch.Tensor:
    """x [heads, dim]: pairs (i, i + dims / 2), i < dims / 2, turned by pos * frequency; the rest unchanged."""
    y, half = x.clone(), dims // 2
    for i in range(half):
        a = pos * rope_frequency(i, dims, base, scaling)
        c, s = math.cos(a), math.sin(a)
        y[:, i] = x[:, i] * c - x[:, i + half] * s
        y[:, i + half] = x[:, i + half] * c + x[:, i] * s
    return y


def window_attention(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, scale: float, window: Optional[int]) -> torch.Tensor:
    """One head: q, k [T, d], v [T, dv]; position i sees the ``window`` positions that end at i; ordinary softmax."""
    T = q.shape[0]
    out = torch.zeros((T, v.shape[1]), dtype=F64)
    for i in range(T):
        lo = max(0, i - window + 1) if window else 0
        s = (k[lo: i + 1] @ q[i]) * scale
        p = torch.exp(s - s.max())
        out[i] = (p / p.sum()) @ v[lo: i + 1]
    return out


# ------------------------------------------------------------------ mixers
def attention(h: torch.Tensor, m: dict, W: Dict[str, torch.Tensor], p: str, eps: float, act_round: Round = None) -> torch.Tensor:
    H, G, d, scale = m["heads"], m["kv_heads"], m["dim"], float(m["scale"])
    rot, mask = m.get("rot"), m.get("mask")
    T = h.shape[0]
    q = (h @ W[p + "q"].T + W[p + "q.b"]).view(T, H, d)
    k = (h @ W[p + "k"].T + W[p + "k.b"]).view(T, G, d)
    v = _r(k.clone(), act_round)
    if rot and rot["dims"]:
        q = torch.stack([rotate_halves(q[t], t, rot["dims"], float(rot["base"]), rot.get("scaling")) for t in range(T)])
        k = torch.stack([rotate_halves(k[t], t, rot["dims"], float(rot["base"]), rot.get("scaling")) for t in range(T)])
    q, k = _r(rms_norm(q, None, eps), act_round), _r(rms_norm(k, None, eps), act_round)
    out = torch.zeros((T, H, d), dtype=F64)
    for n in range(H):
        g = n // (H // G)
        out[:, n] = window_attention(q[:, n], k[:, g], v[:, g], scale, mask["size"] if mask else None)
    gate = sigmoid(h @ W[p + "g"].T)
    return _r(out.reshape(T, H * d) * gate, act_round) @ W[p + "o"].T


def gru_walk(z: torch.Tensor, u: torch.Tensor) -> torch.Tensor:
    """z, u [T, W] -> the state after every token."""
    cand = torch.where(u >= 0, u + 0.5, sigmoid(u))
    S, out = torch.zeros(z.shape[1], dtype=F64), torch.zeros_like(z)
    for t in range(z.shape[0]):
        S = (1.0 - z[t]) * S + z[t] * cand[t]
        out[t] = S
    return out


def mingru(h: torch.Tensor, m: dict, W: Dict[str, torch.Tensor], p: str, act_round: Round = None) -> torch.Tensor:
    z = sigmoid(h @ W[p + "z"].T + W[p + "z.b"])
    u = h @ W[p + "x"].T + W[p + "x.b"]
    return _r(gru_walk(z, u) * silu(h @ W[p + "g"].T), act_round) @ W[p + "o"].T


# ------------------------------------------------------------------ feed-forwards
def gelu_unit(h, W, p, act_round: Round = None):
    return _r(gelu(h @ W[p + "up"].T), act_round) @ W[p + "down"].T


def clamped_unit(h, W, p, limit: float, act_round: Round = None):
    g = torch.clamp(h @ W[p + "gate"].T, max=limit)
    u = torch.clamp(h @ W[p + "up"].T, min=-limit, max=limit)
    return _r(g * sigmoid(GLU_ALPHA * g) * (u + 1.0), act_round) @ W[p + "down"].T


def route(z: torch.Tensor, top: int):
    """z [E] router logits -> (chosen indices, weights): the largest sigmoids (the lower index among equals), as they are."""
    order = sorted(range(z.shape[0]), key=lambda e: (-float(z[e]), e))[:top]
    return order, torch.stack([sigmoid(z[e]) for e in order])


def routed_experts(h: torch.Tensor, mlp: dict, W: Dict[str, torch.Tensor], p: str, act_round: Round = None, choices: Optional[list] = None,
                   margins: Optional[list] = None, chosen: Optional[list] = None) -> torch.Tensor:
    """``choices``: per token the experts to use instead of the router's own choice (weights still from the scores).
    ``chosen`` / ``margins``: lists that receive, per token, the router's own choice and by how much (in logits) its
    last chosen expert beat the best one left out."""
    top, limit = mlp["router"]["top"], float(mlp["expert"]["limit"])
    z = h @ W[p + "router"].T
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        order, _ = route(z[t], top)
        if chosen is not None:
            chosen.append(list(order))
        if margins is not None:
            ranked = sorted((float(v) for v in z[t]), reverse=True)
            margins.append(ranked[top - 1] - ranked[top] if top < len(ranked) else float("inf"))
        if choices is not None:
            order = list(choices[t])
        for e in order:
            out[t] += clamped_unit(_r(sigmoid(z[t, e]) * h[t:t + 1], act_round), W, f"{p}e{e}.", limit, act_round)[0]
    return out


# ------------------------------------------------------------------ the model
def forward(config: dict, W: Dict[str, torch.Tensor], tokens: List[int], act_round: Round = None, streams: Optional[list] = None,
            choices: Optional[dict] = None, margins: Optional[dict] = None, chosen: Optional[dict] = None) -> torch.Tensor:
    """Logits [T, vocab] (float64) of the whole sequence.  ``streams``: a list that receives the sum of the
    streams after every layer.  ``choices``: {layer index: per token the experts to use}; ``margins`` / ``chosen``: dicts
    that receive, per routed layer, what ``routed_experts`` reports."""
    W = {n: t.to(F64) for n, t in W.items()}
    eps = float(config["norm"]["eps"])
    X = [W["embed"][torch.tensor(tokens, dtype=torch.long)] for _ in range(config["streams"])]
    for i, layer in enumerate(config["layers"]):
        p, m, mlp = f"l{i}.", layer["mixer"], layer.get("mlp")

        def reads(q):
            return rms_norm(sum(W[f"{p}hc{q}.in"][s] * x for s, x in enumerate(X)), W[f"{p}norm{q}"], eps)

        h = _r(shift_in(reads(1), W[p + "shift"]), act_round)
        if layer["type"] == "attention":
            y = attention(h, m, W, p + "mix.", eps, act_round)
        elif layer["type"] == "mingru":
            y = mingru(h, m, W, p + "mix.", act_round)
        else:
            raise ValueError(f"unknown layer type {layer['type']}")
        X = mix_streams(X, y, W[p + "hc1.mix"], W[p + "hc1.out"])
        if mlp is not None:
            h = _r(reads(2), act_round)
            if mlp["kind"] == "dense":
                y = gelu_unit(h, W, p + "mlp.", act_round)
            else:
                y = routed_experts(h, mlp, W, p + "mlp.", act_round, None if choices is None else choices.get(i),
                                   None if margins is None else margins.setdefault(i, []), None if chosen is None else chosen.setdefault(i, []))
            X = mix_streams(X, y, W[p + "hc2.mix"], W[p + "hc2.out"])
        if streams is not None:
            streams.append(sum(X))
    h = _r(rms_norm(sum(X), W["final.norm"], eps), act_round)
    return h @ W["head"].T


def greedy(config: dict, W: Dict[str, torch.Tensor], prompt: List[int], new_tokens: int) -> List[int]:
    tokens, out = list(prompt), []
    for _ in range(new_tokens):
        nxt = int(torch.argmax(forward(config, W, tokens)[-1]))
        out.append(nxt)
        tokens.append(nxt)
    return out
