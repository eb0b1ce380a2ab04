"""Arrangements of norm, mixer and feed-forward around the residual stream.

Pre-norm order of the reference (include/photon/arch/transformer_block.hpp:34-51,
src/arch/transformer_block.cpp:189-299):
``x += mixer(norm1(x)); x += ffn(norm2(x))``.
"""
from __future__ import annotations

from typing import Dict, List, Optional, Tuple

import torch

from .. import ops
from ..errors import UnsupportedModelError
from ..weights.loader import TensorSpec
from .base import BLOCKS, MIXERS, Block, FeedForward, LayerCache, Mixer, Norm, Part, StepContext
from .norm import LEFT_JOIN, LEFT_UPDATE, LeftJoin
from .token_shift import TokenShift


class SideBySide(Mixer):
    """Several mixers that read the same input, their results summed into the stream:
    ``x += sum_i scale_i * mixer_i(h)``.  Every mixer keeps a cache or state of its own
    (``mixers()``; ``forward`` takes their ``LayerCache`` in that order) and applies its own
    factor (its ``out_scale``) to its last activation, in float32, before the output projection
    that accumulates into the stream: the sum costs no kernel.

    ``branches``: [(prefix, mixer)]."""

    def __init__(self, branches):
        if not branches:
            raise UnsupportedModelError("mixers side by side: none given")
        self.branches: List[Tuple[str, Mixer]] = list(branches)
        for _, m in self.branches:
            if not getattr(m, "accumulate", True):
                raise UnsupportedModelError(f"{type(m).__name__} must add its result into the stream to stand beside other mixers")

    def mixers(self) -> List[Mixer]:
        return [m for _, m in self.branches]

    def tensor_specs(self) -> List[TensorSpec]:
        return [s.with_prefix(p) for p, m in self.branches for s in m.tensor_specs()]

    def load(self, tensors: Dict[str, torch.Tensor], dtype, device) -> None:
        super().load(tensors, dtype, device)
        for prefix, m in self.branches:
            names = [prefix + s.name for s in m.tensor_specs()]
            m.load({n[len(prefix):]: tensors[n] for n in names}, dtype, device)

    @property
    def graph_safe(self) -> bool:
        return all(m.graph_safe for _, m in self.branches)

    def streamed_weights(self) -> List[torch.Tensor]:
        return [w for _, m in self.branches for w in m.streamed_weights()]

    def forward(self, h: torch.Tensor, x: torch.Tensor, ctx: StepContext, cache) -> None:
        caches = cache if isinstance(cache, (list, tuple)) else [cache]
        for (_, m), c in zip(self.branches, caches):
            m.forward(h, x, ctx, c)


MIXERS.register("side_by_side", SideBySide)


class PreNormBlock(Block):
    """Each of the four parts comes with the name prefix of its tensors inside the block.  The
    mixer may be several side by side (``SideBySide``); ``norm2`` and ``ffn`` None: a layer without
    a feed-forward."""

    def __init__(self, norm1: Tuple[str, Norm], mixer: Tuple[str, Mixer],
                 norm2: Optional[Tuple[str, Norm]] = None, ffn: Optional[Tuple[str, FeedForward]] = None):
        if (ffn is None) != (norm2 is None):
            raise UnsupportedModelError("a feed-forward and its norm come together")
        self._named: List[Tuple[str, Part]] = [norm1, mixer] + ([norm2, ffn] if ffn is not None else [])
        self.norm1, self.mixer = norm1[1], mixer[1]
        self.norm2, self.ffn = (norm2[1], ffn[1]) if ffn is not None else (None, None)

    def mixers(self) -> List[Mixer]:
        inner = getattr(self.mixer, "mixers", None)
        return inner() if inner is not None else [self.mixer]

    def tensor_specs(self) -> List[TensorSpec]:
        return [s.with_prefix(p) for p, part in self._named for s in part.tensor_specs()]

    def load(self, tensors: Dict[str, torch.Tensor], dtype, device) -> None:
        super().load(tensors, dtype, device)
        # a part's tensors: those named by its own list (a prefix may be a prefix of another)
        for prefix, part in self._named:
            names = [prefix + s.name for s in part.tensor_specs()]
            part.load({n[len(prefix):]: tensors[n] for n in names}, dtype, device)

    @property
    def graph_safe(self) -> bool:
        return all(part.graph_safe for _, part in self._named)

    def streamed_weights(self) -> List[torch.Tensor]:
        return [w for _, part in self._named for w in part.streamed_weights()]

    @property
    def reads_deferred(self) -> bool:
        return bool(getattr(self.norm1, "consumes_deferred", False))

    def forward(self, x: torch.Tensor, ctx: StepContext, cache: LayerCache) -> None:
        # A mixer or feed-forward may leave its update of x in pieces (ops.gemm(..., may_defer=True))
        # when the stream's next reader adds them: norm2 after the mixer; after the feed-forward,
        # whoever the model says reads the stream next.
        if self.ffn is None:
            ctx.may_defer = ctx.after_block_consumes
            self.mixer.forward(self.norm1.forward(x, ctx), x, ctx, cache)
            ctx.may_defer = False
            return
        ctx.may_defer = bool(getattr(self.norm2, "consumes_deferred", False))
        self.mixer.forward(self.norm1.forward(x, ctx), x, ctx, cache)
        ctx.may_defer = ctx.after_block_consumes
        self.ffn.forward(self.norm2.forward(x, ctx), x, ctx)
        ctx.may_defer = False


BLOCKS.register("prenorm", PreNormBlock)


class OutputNormBlock(Block):
    """Sublayers that read the stream itself and are normalised on the way out:

        x <- x + mult * norm1(mix(x));   x <- x + mult * norm2(ffn(x))   (no feed-forward: the first only)

    ``mix`` is one mixer, or two side by side that read the same input: then each result is first
    normalised with a weight of its own and the two are averaged.  The norms, the mean, the scaled
    add and the copy of the new stream in the activation type are one kernel per sublayer.  The
    mixers and the feed-forward write their result (``accumulate=False``) instead of adding it.

    ``branches``: [(prefix, mixer, (prefix, norm) or None)]; ``norm1`` / ``norm2`` / ``ffn``: (prefix, part).
    """

    reads_deferred = False
    _STREAM = "stream in the activation type"     # key in ctx.scratch: (stream, its copy) left for the next reader

    def __init__(self, branches, norm1: Tuple[str, Norm], mult: float, norm2=None, ffn=None):
        if not 1 <= len(branches) <= 2:
            raise UnsupportedModelError(f"an output-norm block holds one mixer or two side by side, not {len(branches)}")
        if len(branches) == 2 and any(b[2] is None for b in branches):
            raise UnsupportedModelError("two mixers side by side each need the norm of their result")
        if (ffn is None) != (norm2 is None):
            raise UnsupportedModelError("a feed-forward and its norm come together")
        self.branches = list(branches)
        self.norm1, self.norm2, self.ffn = norm1[1], norm2[1] if norm2 else None, ffn[1] if ffn else None
        self.mult = float(mult)
        self._named: List[Tuple[str, Part]] = [(p, m) for p, m, _ in branches] + [n for _, _, n in branches if n is not None] + [norm1]
        if ffn is not None:
            self._named += [norm2, ffn]
        for _, part in self._named:
            if getattr(part, "accumulate", False):
                raise UnsupportedModelError(f"{type(part).__name__} must be built with accumulate=False inside an output-norm block")

    def mixers(self) -> List[Mixer]:
        return [m for _, m, _ in self.branches]

    def tensor_specs(self) -> List[TensorSpec]:
        return [s.with_prefix(p) for p, part in self._named for s in part.tensor_specs()]

    def load(self, tensors: Dict[str, torch.Tensor], dtype, device) -> None:
        super().load(tensors, dtype, device)
        # a part's tensors: those named by its own list (prefixes here may be prefixes of one another)
        for prefix, part in self._named:
            names = [prefix + s.name for s in part.tensor_specs()]
            part.load({n[len(prefix):]: tensors[n] for n in names}, dtype, device)

    @property
    def graph_safe(self) -> bool:
        return all(part.graph_safe for _, part in self._named)

    def streamed_weights(self) -> List[torch.Tensor]:
        return [w for _, part in self._named for w in part.streamed_weights()]

    def forward(self, x: torch.Tensor, ctx: StepContext, cache) -> None:
        left = ctx.scratch.pop(self._STREAM, None)
        h = left[1] if left is not None and left[0] is x else ops.cast_stream(x, self.dtype)
        caches = cache if isinstance(cache, (list, tuple)) else [cache]
        ctx.may_defer = False
        outs = []
        for (_, mixer, _), c in zip(self.branches, caches):
            out = torch.empty_like(x)
            mixer.forward(h, out, ctx, c)
            outs.append(out)
        norms = [n[1] if n is not None else None for _, _, n in self.branches]
        eps = self.norm1.eps
        if len(outs) == 2:
            h = ops.branch_norm_add(x, outs[0], self.norm1.weight_f32(), eps, self.mult, norms[0].weight_f32(), outs[1],
                                    norms[1].weight_f32(), h_dtype=self.dtype)
        else:
            h = ops.branch_norm_add(x, outs[0], self.norm1.weight_f32(), eps, self.mult,
                                    norms[0].weight_f32() if norms[0] is not None else None, h_dtype=self.dtype)
        if self.ffn is not None:
            out = torch.empty_like(x)
            self.ffn.forward(h, out, ctx)
            h = ops.branch_norm_add(x, out, self.norm2.weight_f32(), self.norm2.eps, self.mult, h_dtype=self.dtype)
        ctx.scratch[self._STREAM] = (x, h)


BLOCKS.register("output_norm", OutputNormBlock)


class SandwichBlock(Block):
    """A norm in front of every sublayer and another behind it:

        x <- x + post1(mix(pre1(x)));   x <- x + post2(ffn(pre2(x)))     (no feed-forward: the first only)

    ``mix`` is one mixer, or two side by side that read the same input: then each result is first RMS-normalised
    over the width with a weight of its own and the two are averaged.  The four norms are layer norms with weight and
    bias (``LayerNorm``).  The branch norms, the mean, the norm behind the sublayer, the add and the norm in front of the
    next sublayer of the block are one kernel.  The mixers and the feed-forward write their result
    (``accumulate=False``) instead of adding it.

    ``branches``: [(prefix, mixer, (prefix, rmsnorm) or None)]; ``pre1`` / ``post1`` / ``pre2`` / ``post2`` / ``ffn``: (prefix, part).
    """

    reads_deferred = False
    NORMS_ARE = ("weight_bias_f32", "layer norms with weight and bias")

    def __init__(self, branches, pre1: Tuple[str, Norm], post1: Tuple[str, Norm], pre2=None, post2=None, ffn=None):
        if not 1 <= len(branches) <= 2:
            raise UnsupportedModelError(f"a sandwich block holds one mixer or two side by side, not {len(branches)}")
        if len(branches) == 2 and any(b[2] is None for b in branches):
            raise UnsupportedModelError("two mixers side by side each need the norm of their result")
        if not ((ffn is None) == (pre2 is None) == (post2 is None)):
            raise UnsupportedModelError("a feed-forward and its two norms come together")
        self.branches = list(branches)
        self.pre1, self.post1 = pre1[1], post1[1]
        self.pre2, self.post2, self.ffn = (pre2[1], post2[1], ffn[1]) if ffn is not None else (None, None, None)
        self._named: List[Tuple[str, Part]] = [pre1, post1] + [(p, m) for p, m, _ in branches] + [n for _, _, n in branches if n is not None]
        if ffn is not None:
            self._named += [pre2, post2, ffn]
        for _, part in [(p, m) for p, m, _ in branches] + ([ffn] if ffn is not None else []):
            if getattr(part, "accumulate", True):
                raise UnsupportedModelError(f"{type(part).__name__} must be built with accumulate=False inside a sandwich block")
        for n in (self.pre1, self.post1, self.pre2, self.post2):
            if n is not None and not hasattr(n, self.NORMS_ARE[0]):
                raise UnsupportedModelError(f"this sandwich block's norms are {self.NORMS_ARE[1]}, not {type(n).__name__}")

    def mixers(self) -> List[Mixer]:
        return [m for _, m, _ in self.branches]

    def tensor_specs(self) -> List[TensorSpec]:
        return [s.with_prefix(p) for p, part in self._named for s in part.tensor_specs()]

    def load(self, tensors: Dict[str, torch.Tensor], dtype, device) -> None:
        super().load(tensors, dtype, device)
        # a part's tensors: those named by its own list (prefixes here may be prefixes of one another)
        for prefix, part in self._named:
            names = [prefix + s.name for s in part.tensor_specs()]
            part.load({n[len(prefix):]: tensors[n] for n in names}, dtype, device)

    @property
    def graph_safe(self) -> bool:
        return all(part.graph_safe for _, part in self._named)

    def streamed_weights(self) -> List[torch.Tensor]:
        return [w for _, part in self._named for w in part.streamed_weights()]

    def forward(self, x: torch.Tensor, ctx: StepContext, cache) -> None:
        caches = cache if isinstance(cache, (list, tuple)) else [cache]
        ctx.may_defer = False
        h = self.pre1.forward(x, ctx)
        outs = []
        for (_, mixer, _), c in zip(self.branches, caches):
            out = torch.empty_like(x)
            mixer.forward(h, out, ctx, c)
            outs.append(out)
        norms = [n[1] if n is not None else None for _, _, n in self.branches]
        nxt = self.pre2.weight_bias_f32() if self.ffn is not None else None
        # a mixer may leave the bias of its last product to this kernel (``pending_bias``)
        a_bias = getattr(self.branches[0][1], "pending_bias", None)
        w_a = norms[0].weight_f32() if norms[0] is not None else None
        if len(outs) == 2:
            h = ops.sandwich_norm_add(x, outs[0], self.post1.weight_bias_f32(), self.post1.eps, nxt, self.dtype, w_a=w_a, b=outs[1],
                                      w_b=norms[1].weight_f32(), a_bias=a_bias)
        else:
            h = ops.sandwich_norm_add(x, outs[0], self.post1.weight_bias_f32(), self.post1.eps, nxt, self.dtype, w_a=w_a, a_bias=a_bias)
        if self.ffn is not None:
            out = torch.empty_like(x)
            self.ffn.forward(h, out, ctx)
            ops.sandwich_norm_add(x, out, self.post2.weight_bias_f32(), self.post2.eps)


BLOCKS.register("sandwich", SandwichBlock)


class RMSSandwichBlock(SandwichBlock):
    """The sandwich with RMS norms (``RMSNorm``) and one mixer:

        x <- x + rms(mix(rms(x; pre1)); post1);   x <- x + rms(ffn(rms(x; pre2)); post2)     (no feed-forward: the first only)

    A sublayer's result joins the stream through its norm, and the next sublayer's input is made, in one kernel; the kernel
    adds the pieces of a product that was split over k, and sums a token's experts, on the way.  The last sublayer's result
    is left to whoever reads the stream next (``LEFT_JOIN``: the next block's first norm, or the final norm)."""

    takes_left_join = True
    NORMS_ARE = ("weight_f32", "RMS norms")

    def __init__(self, branches, pre1: Tuple[str, Norm], post1: Tuple[str, Norm], pre2=None, post2=None, ffn=None):
        if len(branches) != 1 or branches[0][2] is not None:
            raise UnsupportedModelError("a sandwich block with RMS norms holds one mixer")
        super().__init__(branches, pre1, post1, pre2, post2, ffn)

    def forward(self, x: torch.Tensor, ctx: StepContext, cache) -> None:
        h = self.pre1.forward(x, ctx)
        left = self._sublayer(self.branches[0][1], h, x, ctx, self.post1, (cache[0] if isinstance(cache, (list, tuple)) else cache,))
        if self.ffn is not None:
            h = left.apply(ctx.workspace, self.pre2.weight_f32(), self.pre2.eps, self.dtype)
            left = self._sublayer(self.ffn, h, x, ctx, self.post2, ())
        ctx.scratch[LEFT_JOIN] = left

    @staticmethod
    def _sublayer(part: Part, h: torch.Tensor, x: torch.Tensor, ctx: StepContext, post: Norm, cache: tuple) -> LeftJoin:
        y = torch.empty_like(x)
        ctx.may_defer = ctx.may_leave_choices = True
        part.forward(h, y, ctx, *cache)
        ctx.may_defer = ctx.may_leave_choices = False
        choices = ctx.scratch.pop(ops.LEFT_CHOICES, None)
        return LeftJoin(x, y, post.weight_f32(), post.eps, choices if choices is not None and choices.target is y else None)


BLOCKS.register("rms_sandwich", RMSSandwichBlock)


class HyperConnections(Part):
    """How one sublayer is tied to several residual streams side by side (hyper-connections; Zhu et al.,
    "Hyper-Connections"): it reads ``u = sum_s in[s] X_s``, and its result y joins every stream while they mix,
    ``X_t <- sum_s mix[s, t] X_s + out[t] y`` (rows of mix: where from; columns: where to)."""

    graph_safe = True

    def __init__(self, streams: int):
        self.streams = int(streams)
        if not 0 < self.streams <= ops.HYPER_MAX_STREAMS:
            raise UnsupportedModelError(f"{self.streams} residual streams (1 to {ops.HYPER_MAX_STREAMS} are served)")

    def tensor_specs(self) -> List[TensorSpec]:
        n = self.streams
        return [TensorSpec("in", (n,), "norm"), TensorSpec("out", (n,), "norm"), TensorSpec("mix", (n, n), "near_identity")]

    def load(self, tensors: Dict[str, torch.Tensor], dtype, device) -> None:
        super().load(tensors, dtype, device)
        f32 = lambda name: tensors[name].to(torch.float32).reshape(-1)
        self.read = f32("in").contiguous()
        self.post = torch.cat([f32("out"), f32("mix")]).contiguous()      # as the kernel takes them


class HyperConnectionBlock(Block):
    """Pre-norm sublayers on several residual streams side by side (the stream is [T, streams, D]); what the mixer reads
    may be shifted towards the token before (``TokenShift``):

        h = rms(sum_s in1[s] X_s; norm1), shifted;   X_t <- sum_s mix1[s, t] X_s + out1[t] * mixer(h)
        h = rms(sum_s in2[s] X_s; norm2);            X_t <- sum_s mix2[s, t] X_s + out2[t] * ffn(h)     (no feed-forward: the first only)

    The mixer and the feed-forward write their result (``accumulate=False``), or leave it in the pieces of its product.
    A sublayer's update of the streams and the next sublayer's h are one kernel, which reads and writes the streams
    once; the last sublayer's update is left to whoever reads the streams next (the next block's first kernel, or the
    final norm).  The shift is part of that kernel in a step of single tokens, and a kernel of its own in others.

    ``norm1`` / ``mixer`` / ``norm2`` / ``ffn``: (prefix, part); ``shift``: the name of the shift's tensor, or None;
    ``connections``: the prefixes of the two sublayers' ``HyperConnections``."""

    reads_deferred = False

    def __init__(self, hidden_size: int, streams: int, norm1: Tuple[str, Norm], mixer: Tuple[str, Mixer], shift: Optional[str] = None,
                 norm2: Optional[Tuple[str, Norm]] = None, ffn: Optional[Tuple[str, FeedForward]] = None, connections=("hc1.", "hc2.")):
        if (ffn is None) != (norm2 is None):
            raise UnsupportedModelError("a feed-forward and its norm come together")
        for part in [mixer[1]] + ([ffn[1]] if ffn is not None else []):
            if getattr(part, "accumulate", True):
                raise UnsupportedModelError(f"{type(part).__name__} must be built with accumulate=False between streams side by side")
        self.norm1, self.mixer = norm1[1], mixer[1]
        self.norm2, self.ffn = (norm2[1], ffn[1]) if ffn is not None else (None, None)
        self.shift = TokenShift(hidden_size, tensor_name="") if shift is not None else None
        self.hc1, self.hc2 = HyperConnections(streams), HyperConnections(streams) if ffn is not None else None
        self._named: List[Tuple[str, Part]] = [norm1, mixer, (connections[0], self.hc1)]
        if shift is not None:
            self._named.append((shift, self.shift))
        if ffn is not None:
            self._named += [norm2, ffn, (connections[1], self.hc2)]

    def mixers(self) -> List[Part]:
        return [self.mixer] + ([self.shift] if self.shift is not None else [])

    def tensor_specs(self) -> List[TensorSpec]:
        return [s.with_prefix(p) for p, part in self._named for s in part.tensor_specs()]

    def load(self, tensors: Dict[str, torch.Tensor], dtype, device) -> None:
        super().load(tensors, dtype, device)
        for prefix, part in self._named:
            names = [prefix + s.name for s in part.tensor_specs()]
            part.load({n[len(prefix):]: tensors[n] for n in names}, dtype, device)

    @property
    def graph_safe(self) -> bool:
        return all(part.graph_safe for _, part in self._named)

    def streamed_weights(self) -> List[torch.Tensor]:
        return [w for _, part in self._named for w in part.streamed_weights()]

    def forward(self, x: torch.Tensor, ctx: StepContext, cache) -> None:
        caches = cache if isinstance(cache, (list, tuple)) else [cache]
        ws, reads = ctx.workspace, (self.hc1.read, self.norm1.weight_f32(), self.norm1.eps)
        left = ctx.scratch.pop(LEFT_UPDATE, None)
        y, post = (left[1], left[2]) if left is not None and left[0] is x else (None, None)
        if self.shift is None:
            h = self._join_and_read(x, y, post, self.dtype, reads, ws)
        elif ctx.all_decode:
            h = self._join_and_read(x, y, post, self.dtype, reads, ws, shift=self.shift.share, state=caches[1].state, ctx=ctx)
        else:
            h = ops.token_shift(self._join_and_read(x, y, post, torch.float32, reads, ws), self.shift.share, caches[1].state, ctx, self.dtype)
        ctx.may_defer = True                          # the next kernel on the streams adds a product's pieces
        y = self._result(x)
        self.mixer.forward(h, y, ctx, caches[0])
        post = self.hc1.post
        if self.ffn is not None:
            h = self._join_and_read(x, y, post, self.dtype, (self.hc2.read, self.norm2.weight_f32(), self.norm2.eps), ws)
            y = self._result(x)
            self.ffn.forward(h, y, ctx)
            post = self.hc2.post
        ctx.may_defer = False
        ctx.scratch[LEFT_UPDATE] = (x, y, post)

    @staticmethod
    def _join_and_read(x, y, post, dtype, reads, ws, **kw):
        read, norm, eps = reads
        return ops.hyper_streams(x, y=y, post=post, h_dtype=dtype, read=read, norm=norm, eps=eps, ws=ws, **kw)

    @staticmethod
    def _result(x: torch.Tensor) -> torch.Tensor:
        return torch.empty((x.shape[0], x.shape[2]), dtype=torch.float32, device=x.device)


BLOCKS.register("hyper_connections", HyperConnectionBlock)
