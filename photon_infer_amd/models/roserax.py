"""Roserax: a decoder whose every sublayer sits between two RMS norms, with three kinds of mixer - attention within a window
that keeps a sequence's first tokens, attention through a latent with a gate per feature, retention - and feed-forwards that
are dense (squared relu) or routed; a scaled embedding and a tied head whose logits carry a factor.

    x = embed[token] * scale
    per layer:  x <- x + rms(mixer(rms(x; norm1)); norm1b);  x <- x + rms(ff(rms(x; norm2)); norm2b)   (layers with a feed-forward)
    logits = logit_scale * embed . rms(x; final.norm)

    mixer of an "attention" layer:         no positions in the scores; queries and keys normalised per head with one weight for
                                           all heads; the softmax has a one in its denominator
    mixer of a "latent_attention" layer:   a rotated key part for all heads (paired halves), gates per feature
    mixer of a "retention" layer:          a matrix state per head with a fixed decay

The names of layer i's tensors begin with ``l<i>.``; the mixer's with ``mix.``, the feed-forward's with ``mlp.``; norms are named by themselves
(``l<i>.norm1``, ``final.norm``); the head is the embedding's table.
"""
from __future__ import annotations

from ..config.roserax import GatedLatentAttentionConfig, KeptWindowAttentionConfig, RetentionConfig, RoseraxConfig
from ..errors import UnsupportedModelError
from ..parts import BLOCKS, FEED_FORWARDS, MIXERS, NORMS, POSITION_ENCODINGS
from ..parts.embedding import LMHead, TokenEmbedding
from ..parts.model import ModelSpec
from ..registry import register_architecture


def _mixer(cfg: RoseraxConfig, m, ropes: dict):
    D, eps = cfg.width, cfg.norm_eps

    def rotation(head_dim: int, rot):
        if rot is None:
            return None
        key = (rot.dims, rot.base)
        if key not in ropes:      # layers that rotate alike share the part, and with it a step's table of cosines and sines
            ropes[key] = POSITION_ENCODINGS.make("rope", head_dim=head_dim, theta=rot.base, rotary_dim=rot.dims)
        return ropes[key]

    if isinstance(m, KeptWindowAttentionConfig):
        return MIXERS.make("sink_window_attention", hidden_size=D, num_heads=m.heads, num_kv_heads=m.kv_heads, head_dim=m.dim,
                           value_dim=m.vdim, scale=m.scale, window=m.window, keep_first=m.keep_first, eps=eps, norm_per_head=True,
                           norm_shared=True, distance_bias=False, sink_score=0.0, output_gate=False, accumulate=False)
    if isinstance(m, GatedLatentAttentionConfig):
        return MIXERS.make("latent_attention", hidden_size=D, num_heads=m.heads, head_dim=m.dim, rot_dim=m.rot_dim, value_dim=m.vdim,
                           q_rank=m.q_rank, kv_rank=m.kv_rank, scale=m.scale, eps=eps, position=rotation(m.rot_dim, m.rot), gate="g",
                           accumulate=False)
    if isinstance(m, RetentionConfig):
        return MIXERS.make("retention", hidden_size=D, num_heads=m.heads, key_dim=m.dim, value_dim=m.vdim, decays=m.decay, eps=eps,
                           position=rotation(m.dim, m.rot), accumulate=False)
    raise UnsupportedModelError(f"no mixer for {type(m).__name__}")


def _feed_forward(cfg: RoseraxConfig, mlp):
    if mlp.kind == "dense":
        return FEED_FORWARDS.make("squared_relu_mlp", hidden_size=cfg.width, intermediate_size=mlp.ff, accumulate=False)
    return FEED_FORWARDS.make("routed_experts", hidden_size=cfg.width, expert_size=mlp.ff, num_experts=mlp.experts, top=mlp.top,
                              groups=mlp.groups, keep=mlp.keep, accumulate=False)


def build_roserax(cfg: RoseraxConfig) -> ModelSpec:
    D, eps = cfg.width, cfg.norm_eps
    norm = lambda: NORMS.make("rmsnorm", dim=D, eps=eps, tensor_name="")
    layers, ropes, ignorable = [], {}, []
    for i, layer in enumerate(cfg.layers):
        pre2 = post2 = ffn = None
        if layer.mlp is not None:
            pre2, post2, ffn = ("norm2", norm()), ("norm2b", norm()), ("mlp.", _feed_forward(cfg, layer.mlp))
        else:
            ignorable += [f"l{i}.norm2", f"l{i}.norm2b"]       # a layer without feed-forward has no use for its norms
        layers.append((f"l{i}.", BLOCKS.make("rms_sandwich", branches=[("mix.", _mixer(cfg, layer.mixer, ropes), None)], pre1=("norm1", norm()),
                                             post1=("norm1b", norm()), pre2=pre2, post2=post2, ffn=ffn)))
    # the factor on the logits is made part of the final norm's weight: the head is a plain product
    return ModelSpec(
        hidden_size=D, vocab_size=cfg.vocab, max_positions=cfg.max_positions,
        embedding=("embed", TokenEmbedding(cfg.vocab, D, tensor_name="", scale=cfg.embedding_scale)), layers=layers,
        final_norm=("final.norm", NORMS.make("rmsnorm", dim=D, eps=eps, tensor_name="", mult=cfg.logit_scale)),
        head=("head", LMHead(cfg.vocab, D, tied=True, tensor_name="")), ignorable=tuple(ignorable),
    )


register_architecture("Roserax", RoseraxConfig, build_roserax)
