"""Semezen: a decoder with several residual streams side by side.  Every sublayer reads a weighted sum of them and
writes to all of them through a small matrix; a token's mixer also sees the token before it; mixers are windowed
attention whose values are its keys, or minGRU, a recurrence of one number per feature; feed-forwards are
dense (gelu) or routed.

    X_s = embed[token]   (s = 1 .. streams)
    per layer, q = 1 (the mixer), 2 (the feed-forward, where there is one):
        h = rms(sum_s in_q[s] X_s; norm_q);   for the mixer  h <- h + (h of the token before - h) * shift
        X_t <- sum_s mix_q[s, t] X_s + out_q[t] * sublayer(h)
    logits = head . rms(sum_s X_s; final.norm)

The names of layer i's tensors begin with ``l<i>.``: ``norm1`` / ``norm2``, ``shift``, ``hc1.`` / ``hc2.`` (in, out, mix), ``mix.`` (the
mixer) and ``mlp.``.
"""
from __future__ import annotations

from ..config.semezen import MinGruConfig, SemezenConfig, WindowAttentionConfig
from ..errors import UnsupportedModelError
from ..parts import BLOCKS, FEED_FORWARDS, MIXERS, NORMS, POSITION_ENCODINGS
from ..parts.embedding import LMHead, TokenEmbedding
from ..parts.model import ModelSpec
from ..registry import register_architecture

GLU_ALPHA = 1.702      # the factor inside the experts' gate sigmoid; the design fixes it


def _mixer(cfg: SemezenConfig, m, ropes: dict):
    D = cfg.width
    if isinstance(m, MinGruConfig):
        return MIXERS.make("min_gru", hidden_size=D, width=m.width, accumulate=False)
    if isinstance(m, WindowAttentionConfig):
        rope = None
        if m.rot_dims:
            # layers that rotate alike share the part, and with it a step's table of cosines and sines
            key = (m.dim, m.rot_dims, m.rot_base, m.rot_scaling)
            if key not in ropes:
                ropes[key] = POSITION_ENCODINGS.make("rope", head_dim=m.dim, theta=m.rot_base, scaling=m.rot_scaling, rotary_dim=m.rot_dims)
            rope = ropes[key]
        return MIXERS.make("attention", hidden_size=D, num_heads=m.heads, num_kv_heads=m.kv_heads, head_dim=m.dim, position=rope,
                           scale=m.scale, window=m.window, names=("q", "k", "v", "o"), any_head_size=True, qkv_bias=True, accumulate=False,
                           values_are_keys=True, head_norm_eps=cfg.norm_eps, feature_gate="g")
    raise UnsupportedModelError(f"no mixer for {type(m).__name__}")


def _feed_forward(cfg: SemezenConfig, mlp):
    D = cfg.width
    if mlp.kind == "dense":
        return FEED_FORWARDS.make("gelu_mlp", hidden_size=D, intermediate_size=mlp.ff, accumulate=False)
    return FEED_FORWARDS.make("routed_experts", hidden_size=D, expert_size=mlp.ff, num_experts=mlp.experts, top=mlp.top, scoring="sigmoid",
                              weigh_input=True, activation="clamped_glu", limit=mlp.limit, alpha=GLU_ALPHA, accumulate=False)


def build_semezen(cfg: SemezenConfig) -> ModelSpec:
    D, S, eps = cfg.width, cfg.streams, cfg.norm_eps
    norm = lambda: NORMS.make("rmsnorm", dim=D, eps=eps, tensor_name="")
    layers, ropes, ignorable = [], {}, []
    for i, layer in enumerate(cfg.layers):
        norm2 = ffn = None
        if layer.mlp is not None:
            norm2, ffn = ("norm2", norm()), ("mlp.", _feed_forward(cfg, layer.mlp))
        else:
            ignorable += [f"l{i}.norm2", f"l{i}.hc2.*"]       # a layer without feed-forward has no use for them
        layers.append((f"l{i}.", BLOCKS.make("hyper_connections", hidden_size=D, streams=S, norm1=("norm1", norm()),
                                             mixer=("mix.", _mixer(cfg, layer.mixer, ropes)), shift="shift", norm2=norm2, ffn=ffn,
                                             connections=("hc1.", "hc2."))))
    return ModelSpec(
        hidden_size=D, vocab_size=cfg.vocab, max_positions=cfg.max_positions,
        embedding=("", TokenEmbedding(cfg.vocab, D, tensor_name="embed", copies=S)), layers=layers,
        final_norm=("final.norm", NORMS.make("stream_sum_rmsnorm", dim=D, eps=eps, streams=S, tensor_name="")),
        head=("head", LMHead(cfg.vocab, D, tied=False, tensor_name="")), ignorable=tuple(ignorable),
    )


register_architecture("Semezen", SemezenConfig, build_semezen)
