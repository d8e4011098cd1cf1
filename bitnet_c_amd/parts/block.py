"""Arrangement of the parts of one layer.

"prenorm": x += mixer(norm(x)); x += ffn(norm(x)) -- the order of the reference's layer
(src/transformer/cpu.c:536-939 and :1247-1303): norm, mixer, add, norm, feed-forward, add.
A layer without a feed-forward (ffn None; ffn_norm None with it) is the first half alone.
With output norms (mixer_out_norm, ffn_out_norm) a half's output goes through a norm of its own before it joins the
stream: x += norm_out(mixer(norm(x))).  The stream holds such an output back with its norm (NormedDelta), and the
kernel of the next norm forms the normed output, the sum and the next half's input in one pass.

"parallel_prenorm": x += mixer(norm_1(x)) + ffn(norm_2(x)) -- both halves read the same stream, each under a norm of its own,
and their outputs join it together; without a feed-forward the mixer's half alone.

"postnorm": x <- norm(alpha x + gain mixer(x)); x <- norm(alpha x + gain ffn(x)) -- the norms stand behind the sums and
their output is the stream; the halves read the stream itself.  alpha is a constant; with layer_scale every half's output
has weights of its own (gain, one number per column); with token_shift the mixer reads the stream mixed with the previous
token's (parts/shift.py), whose row is part of a sequence's state, beside whatever state the mixer keeps."""
from __future__ import annotations

from dataclasses import replace

import torch

from .base import (BLOCKS, FEED_FORWARDS, MIXERS, NORMS, CacheNeed, JoinedDelta, LazyDelta, NormedDelta, ParamSpec, Part,
                   PartSpec, PostNormedDelta, StateNeed)
from .linear import upload
from .shift import TokenShift


@BLOCKS.register("prenorm")
class PreNormBlock(Part):
    def __init__(self, mixer: PartSpec, ffn: PartSpec | None, mixer_norm: PartSpec, ffn_norm: PartSpec | None = None,
                 mixer_out_norm: PartSpec | None = None, ffn_out_norm: PartSpec | None = None):
        if (ffn is None) != (ffn_norm is None):
            raise ValueError("prenorm block: a feed-forward and its norm come together or not at all")
        if ffn is None and ffn_out_norm is not None:
            raise ValueError("prenorm block: an output norm of a feed-forward that is not there")
        self.mixer = MIXERS.build(mixer)
        self.ffn = FEED_FORWARDS.build(ffn) if ffn is not None else None
        self.mixer_norm = NORMS.build(mixer_norm)
        self.ffn_norm = NORMS.build(ffn_norm) if ffn_norm is not None else None
        self.mixer_out_norm = NORMS.build(mixer_out_norm) if mixer_out_norm is not None else None
        self.ffn_out_norm = NORMS.build(ffn_out_norm) if ffn_out_norm is not None else None
        for n in (self.mixer_out_norm, self.ffn_out_norm):
            if n is not None and not getattr(n, "normed_delta", False):
                raise ValueError("prenorm block: an output norm must be one that the stream can apply to a held-back output")

    @property
    def prompt_capturable(self) -> bool:
        return all(getattr(c, "prompt_capturable", False) for c in self.children().values())

    def children(self):
        c = {"mixer": self.mixer, "ffn": self.ffn, "mixer_norm": self.mixer_norm, "ffn_norm": self.ffn_norm,
             "mixer_out_norm": self.mixer_out_norm, "ffn_out_norm": self.ffn_out_norm}
        return {k: v for k, v in c.items() if v is not None}

    def linears(self):
        return [l for part in self.children().values() for l in getattr(part, "linears", list)()]

    def tensors(self):
        return {f"{cn}.{tn}": spec for cn, c in self.children().items() for tn, spec in c.tensors().items()}

    def load(self, tensors, device, dtype):
        for cn, c in self.children().items():
            c.load({k[len(cn) + 1:]: v for k, v in tensors.items() if k.startswith(cn + ".")}, device, dtype)

    def cache_need(self):
        return self.mixer.cache_need()

    def forward(self, stream, ctx, kv):
        # A part that says so may get its norm undone (it applies it inside its first product) and may hand
        # its last product in undone (it then adds itself to the stream): see ResidualStream.
        tap = getattr(ctx, "tap", None)        # diagnostics (StepContext.tap): the stream at the reference's three dump points
        if tap is not None:
            tap("layer_in", ctx.entry, stream, ctx)
        h = stream.normed(self.mixer_norm, ctx.act_dtype, consumer=self.mixer, ctx=ctx)
        if self.mixer_out_norm is not None:
            stream.add(NormedDelta(self.mixer.forward(h, ctx, kv), self.mixer_out_norm))
        elif getattr(self.mixer, "gives_lazy_delta", False):
            stream.add(self.mixer.forward(h, ctx, kv, lazy_ok=True))
        else:
            stream.add(self.mixer.forward(h, ctx, kv))
        if tap is not None:
            tap("ffn_in", ctx.entry, stream, ctx)
        if self.ffn is None:
            if tap is not None:
                tap("layer_out", ctx.entry, stream, ctx)
            return
        h = stream.normed(self.ffn_norm, ctx.act_dtype, consumer=self.ffn, ctx=ctx)
        if self.ffn_out_norm is not None:
            stream.add(NormedDelta(self.ffn.forward(h, ctx), self.ffn_out_norm))
        elif getattr(self.ffn, "gives_lazy_delta", False):
            stream.add(self.ffn.forward(h, ctx, lazy_ok=True))
        else:
            stream.add(self.ffn.forward(h, ctx))
        if tap is not None:
            tap("layer_out", ctx.entry, stream, ctx)


@BLOCKS.register("parallel_prenorm")
class ParallelPreNormBlock(PreNormBlock):
    """The tensors and children of a pre-norm block; one kernel adds the last block's outputs and forms both norms."""

    def __init__(self, mixer: PartSpec, ffn: PartSpec | None, mixer_norm: PartSpec, ffn_norm: PartSpec | None = None):
        super().__init__(mixer, ffn, mixer_norm, ffn_norm)

    @staticmethod
    def _run(part, *args):
        return part.forward(*args, lazy_ok=True) if getattr(part, "gives_lazy_delta", False) else part.forward(*args)

    def forward(self, stream, ctx, kv):
        tap = getattr(ctx, "tap", None)        # diagnostics; both halves read the stream of "layer_in"
        if tap is not None:
            tap("layer_in", ctx.entry, stream, ctx)
            tap("ffn_in", ctx.entry, stream, ctx)
        if self.ffn is None:
            stream.add(JoinedDelta([self._run(self.mixer, stream.normed(self.mixer_norm, ctx.act_dtype), ctx, kv)]))
        else:
            h_mixer, h_ffn = stream.normed_twice(self.mixer_norm, self.ffn_norm, ctx.act_dtype)
            stream.add(JoinedDelta([self._run(self.mixer, h_mixer, ctx, kv), self._run(self.ffn, h_ffn, ctx)]))
        if tap is not None:
            tap("layer_out", ctx.entry, stream, ctx)


@BLOCKS.register("postnorm")
class PostNormBlock(Part):
    def __init__(self, hidden: int, mixer: PartSpec, ffn: PartSpec | None, mixer_norm: PartSpec, ffn_norm: PartSpec | None = None,
                 alpha: float = 1.0, layer_scale: bool = False, token_shift: bool = False):
        if (ffn is None) != (ffn_norm is None):
            raise ValueError("postnorm block: a feed-forward and its norm come together or not at all")
        self.hidden, self.alpha, self.layer_scale = int(hidden), float(alpha), bool(layer_scale)
        self.mixer = MIXERS.build(mixer)
        self.ffn = FEED_FORWARDS.build(ffn) if ffn is not None else None
        self.mixer_norm = NORMS.build(mixer_norm)
        self.ffn_norm = NORMS.build(ffn_norm) if ffn_norm is not None else None
        for n in (self.mixer_norm, self.ffn_norm):
            if n is not None and not getattr(n, "normed_delta", False):
                raise ValueError("postnorm block: a norm behind a sum is one of RMSNorm's form (weight and eps)")
        self.shift = TokenShift(hidden) if token_shift else None
        self.rows = NORMS.build(PartSpec.of("none", dim=hidden))          # the halves read the stream's rows as they are
        self.mixer_gain = self.ffn_gain = None
        state = self.mixer.cache_need().state
        if self.shift is not None and state is not None and (
                len(state.shape) != 1 or state.dtype != torch.float32 or not state.device_addressed):
            raise ValueError("postnorm block: a token shift's row lies behind a mixer's state of one dimension, float32 and "
                             f"addressed by the device's slot ids, not {state}")
        self.mixer_state = state.shape[0] if state is not None and self.shift is not None else 0

    @property
    def prompt_capturable(self) -> bool:
        return all(getattr(c, "prompt_capturable", False) for c in self.children().values())

    def children(self):
        c = {"mixer": self.mixer, "ffn": self.ffn, "mixer_norm": self.mixer_norm, "ffn_norm": self.ffn_norm, "shift": self.shift}
        return {k: v for k, v in c.items() if v is not None}

    def linears(self):
        return [l for part in self.children().values() for l in getattr(part, "linears", list)()]

    def tensors(self):
        t = {f"{cn}.{tn}": spec for cn, c in self.children().items() for tn, spec in c.tensors().items()}
        if self.layer_scale:
            t["mixer_gain"] = ParamSpec((self.hidden,), "ones")
            if self.ffn is not None:
                t["ffn_gain"] = ParamSpec((self.hidden,), "ones")
        return t

    def load(self, tensors, device, dtype):
        for cn, c in self.children().items():
            c.load({k[len(cn) + 1:]: v for k, v in tensors.items() if k.startswith(cn + ".")}, device, dtype)
        if self.layer_scale:
            self.mixer_gain = upload(tensors["mixer_gain"], device, torch.float32)
            if self.ffn is not None:
                self.ffn_gain = upload(tensors["ffn_gain"], device, torch.float32)

    def cache_need(self):
        need = self.mixer.cache_need()
        if self.shift is None:
            return need
        # the mixer's own state, then the last row of the stream in front of the mixer
        return CacheNeed(kv=need.kv, state=StateNeed((self.mixer_state + self.shift.state_floats,), torch.float32,
                                                     device_addressed=True))

    @staticmethod
    def _run(part, *args):
        """A half's output, a tensor or partial sums: what the stream's kernel adds up itself."""
        if not getattr(part, "gives_lazy_delta", False):
            return part.forward(*args)
        y = part.forward(*args, lazy_ok=True)
        return y.compute() if isinstance(y, LazyDelta) else y

    def forward(self, stream, ctx, kv):
        tap = getattr(ctx, "tap", None)        # diagnostics, at the points of the other blocks
        if tap is not None:
            tap("layer_in", ctx.entry, stream, ctx)
        if self.shift is not None:
            h = self.shift.apply(stream, kv.state[:, self.mixer_state:], ctx)
            kv = replace(kv, state=kv.state[:, :self.mixer_state] if self.mixer_state else None)
        else:
            h = stream.normed(self.rows, ctx.act_dtype)
        stream.add(PostNormedDelta(self._run(self.mixer, h, ctx, kv), self.mixer_norm, self.alpha, self.mixer_gain))
        if tap is not None:
            tap("ffn_in", ctx.entry, stream, ctx)
        if self.ffn is not None:
            h = stream.normed(self.rows, ctx.act_dtype)
            stream.add(PostNormedDelta(self._run(self.ffn, h, ctx), self.ffn_norm, self.alpha, self.ffn_gain))
        if tap is not None:
            tap("layer_out", ctx.entry, stream, ctx)
