"""Arrangement of a layer's parts around the residual stream.

Pre-norm (src/engine.cpp:137-239): h += mixer(norm1(h)); h += ffn(norm2(h)). The
residual stream h is 32-bit; mixer and feed-forward add their result into it
(their last product accumulates into h), so the sum is made in 32-bit.
"""
from __future__ import annotations

import torch

from .. import ops
from .base import Block, FeedForward, Mixer, Norm, ParamSpec
from .registry import register_part
from .token_input import TokenInput


class PreNormBlock(Block):
    graph_safe = True

    def __init__(self, mixer: Mixer, feed_forward: FeedForward | None, mixer_norm: Norm, ffn_norm: Norm | None,
                 names: dict | None = None):
        self.mixer, self.feed_forward = mixer, feed_forward
        self.mixer_norm, self.ffn_norm = mixer_norm, ffn_norm
        # Names under which a checkpoint stores this layer's parts.
        self.names = {"mixer_norm": "input_layernorm", "mixer": "self_attn",
                      "ffn_norm": "post_attention_layernorm", "feed_forward": "mlp"}
        if names:
            self.names.update(names)

    def children(self):
        n = self.names
        out = {n["mixer_norm"]: self.mixer_norm, n["mixer"]: self.mixer}
        if self.feed_forward is not None:
            out.update({n["ffn_norm"]: self.ffn_norm, n["feed_forward"]: self.feed_forward})
        return out

    def forward(self, h, step, cache, write_cache=True):
        T, H = h.shape
        x = step.buffer("block.normed", (T, H), step.act_dtype)
        if self.mixer.fuses_norm(h, self.mixer_norm, step):
            self.mixer.forward(h, step, cache, h, True, write_cache, pre_norm=self.mixer_norm)
        else:
            self.mixer_norm.forward(h, x)
            self.mixer.forward(x, step, cache, h, True, write_cache)
        if self.feed_forward is None:
            return
        if self.feed_forward.fuses_norm(h, self.ffn_norm, step):
            self.feed_forward.forward(h, step, h, True, pre_norm=self.ffn_norm)
        else:
            self.ffn_norm.forward(h, x)
            self.feed_forward.forward(x, step, h, True)


class SandwichBlock(Block):
    """A norm in front of and behind every sublayer: h += post1(mixer(pre1(h))); h += post2(ffn(pre2(h))).
    A sublayer's result is a 32-bit buffer of its own; the norm behind it, the sum into the stream and the
    norm in front of whatever reads the stream next (this block's feed-forward, or the first sublayer of
    the block behind) are one kernel where all three norms are the plain RMS formula."""
    graph_safe = True

    def __init__(self, mixer: Mixer, feed_forward: FeedForward | None, mixer_norm: Norm, ffn_norm: Norm | None,
                 mixer_post_norm: Norm, ffn_post_norm: Norm | None, names: dict | None = None):
        self.mixer, self.feed_forward = mixer, feed_forward
        self.mixer_norm, self.ffn_norm = mixer_norm, ffn_norm
        self.mixer_post_norm, self.ffn_post_norm = mixer_post_norm, ffn_post_norm
        self.names = {"mixer_norm": "norm1", "mixer": "mix", "mixer_post_norm": "norm1b",
                      "ffn_norm": "norm2", "feed_forward": "mlp", "ffn_post_norm": "norm2b"}
        if names:
            self.names.update(names)
        # the block that runs behind this one (told by the model as it runs its schedule; None: unknown)
        self.next_block = None

    def children(self):
        n = self.names
        out = {n["mixer_norm"]: self.mixer_norm, n["mixer_post_norm"]: self.mixer_post_norm, n["mixer"]: self.mixer}
        if self.feed_forward is not None:
            out.update({n["ffn_norm"]: self.ffn_norm, n["ffn_post_norm"]: self.ffn_post_norm,
                        n["feed_forward"]: self.feed_forward})
        return out

    def _join(self, y, post: Norm, h, nxt: Norm | None, x, step) -> bool:
        """h += post(y); True if x was also made = nxt(h)."""
        rms = post.fused_rms()
        nxt_rms = nxt.fused_rms() if nxt is not None else None
        if rms is not None and nxt_rms is not None and nxt_rms[0].dtype == rms[0].dtype and nxt_rms[1] == rms[1]:
            ops.norm_add(y, rms[0], h, rms[1], nxt_rms[0], x)
            return True
        if rms is not None:
            ops.norm_add(y, rms[0], h, rms[1])
        else:
            raise NotImplementedError("sandwich blocks take norms of the plain RMS formula behind their sublayers")
        return False

    def forward(self, h, step, cache, write_cache=True):
        T, H = h.shape
        x = step.buffer("block.normed", (T, H), step.act_dtype)
        y = step.buffer("block.sublayer", (T, H), torch.float32)
        if step.extra.pop("block.normed is for", None) != id(self):
            self.mixer_norm.forward(h, x)
        self.mixer.forward(x, step, cache, y, False, write_cache)
        behind = self.next_block.mixer_norm if isinstance(self.next_block, SandwichBlock) else None
        if self.feed_forward is None:
            if self._join(y, self.mixer_post_norm, h, behind, x, step):
                step.extra["block.normed is for"] = id(self.next_block)
            return
        if not self._join(y, self.mixer_post_norm, h, self.ffn_norm, x, step):
            self.ffn_norm.forward(h, x)
        self.feed_forward.forward(x, step, y, False)
        if self._join(y, self.ffn_post_norm, h, behind, x, step):
            step.extra["block.normed is for"] = id(self.next_block)


class ParallelBlock(Block):
    """One norm whose output both sublayers read: h += mixer(norm(h)) + ffn(norm(h)). Both sublayers add into the
    32-bit stream (their last products accumulate), the mixer first."""
    graph_safe = True

    def __init__(self, mixer: Mixer, feed_forward: FeedForward | None, mixer_norm: Norm, ffn_norm: Norm | None = None,
                 names: dict | None = None):
        if ffn_norm is not None:
            raise ValueError("a parallel block has one norm: its feed-forward reads the mixer's")
        self.mixer, self.feed_forward, self.mixer_norm = mixer, feed_forward, mixer_norm
        self.names = {"mixer_norm": "norm1", "mixer": "mix", "feed_forward": "mlp"}
        if names:
            self.names.update(names)

    def children(self):
        n = self.names
        out = {n["mixer_norm"]: self.mixer_norm, n["mixer"]: self.mixer}
        if self.feed_forward is not None:
            out[n["feed_forward"]] = self.feed_forward
        return out

    def forward(self, h, step, cache, write_cache=True):
        T, H = h.shape
        x = step.buffer("block.normed", (T, H), step.act_dtype)
        self.mixer_norm.forward(h, x)
        self.mixer.forward(x, step, cache, h, True, write_cache)
        if self.feed_forward is not None:
            self.feed_forward.forward(x, step, h, True)


class OutputNormBlock(Block):
    """Norms behind the sublayers only: h += c norm1(mixer(h)); h += c norm2(ffn(h)) with a constant c (`residual_scale`, 1
    unless given). `layer_scale`: what a sublayer adds is multiplied entry by entry by a vector of its own ("ls1", "ls2"; made
    part of the norm's weight, a 32-bit product, when the tensors are loaded). `token_input`: a third sublayer behind the
    other two, the layer's own input from the token's id, normed and added the same way without scale or vector. The sublayers read the stream itself
    (rounded to the activation type where that is not 32-bit); a sublayer's result is a 32-bit buffer of its own, and
    the norm behind it, the sum into the stream and the copy of the updated rows that the next sublayer reads (this
    block's feed-forward, or the mixer of the block behind) are one kernel."""
    graph_safe = True
    ADDED_ROWS = 64             # steps of up to this many rows add the parts of a sublayer's last product

    def __init__(self, mixer: Mixer, feed_forward: FeedForward | None, mixer_norm: Norm, ffn_norm: Norm | None,
                 names: dict | None = None, residual_scale: float = 1.0, layer_scale: bool = False,
                 token_input: TokenInput | None = None):
        self.mixer, self.feed_forward = mixer, feed_forward
        self.mixer_norm, self.ffn_norm = mixer_norm, ffn_norm
        self.residual_scale = float(residual_scale)
        self.layer_scale, self.token_input = bool(layer_scale), token_input
        self.scales: list[torch.Tensor] = []
        self.names = {"mixer_norm": "norm1", "mixer": "mix", "ffn_norm": "norm2", "feed_forward": "mlp", "mixer_scale": "ls1",
                      "ffn_scale": "ls2", "token_input": "side"}
        if names:
            self.names.update(names)
        # the block that runs behind this one (told by the model as it runs its schedule; None: unknown)
        self.next_block = None

    def children(self):
        n = self.names
        out = {n["mixer_norm"]: self.mixer_norm, n["mixer"]: self.mixer}
        if self.feed_forward is not None:
            out.update({n["ffn_norm"]: self.ffn_norm, n["feed_forward"]: self.feed_forward})
        if self.token_input is not None:
            out[n["token_input"]] = self.token_input
        return out

    def _scaled_norms(self) -> list[tuple[str, Norm]]:
        n = self.names
        out = [(n["mixer_scale"], self.mixer_norm)]
        return out + [(n["ffn_scale"], self.ffn_norm)] if self.feed_forward is not None else out

    def param_specs(self):
        if not self.layer_scale:
            return {}
        return {name: ParamSpec((norm.size,), "norm") for name, norm in self._scaled_norms()}

    def load_tree(self, get, placement, prefix=""):
        super().load_tree(get, placement, prefix)
        if self.layer_scale:
            f32 = torch.float32
            self.scales = [placement.place(get(prefix + name), f32) * norm.fused_rms()[0].to(f32) for name, norm in self._scaled_norms()]

    def _join(self, y, post: Norm, h, x, clear: bool, c: float = 1.0, weight: torch.Tensor | None = None) -> None:
        """h += c post(y), and x = the updated rows where x is another buffer than the stream; weight: in place of the norm's
        (its product with the sublayer's vector)."""
        rms = post.fused_rms()
        if rms is None:
            raise NotImplementedError("output-norm blocks take norms of the plain RMS formula behind their sublayers")
        ops.norm_add(y, rms[0] if weight is None else weight, h, rms[1], None, x if x is not h else None, c, clear)

    def forward(self, h, step, cache, write_cache=True):
        T, H = h.shape
        # few rows: a sublayer's last product is cut over k and its parts are added (atomics) into a buffer of zeros, which
        # the norm behind it leaves as zeros again; otherwise it is stored
        add = T <= self.ADDED_ROWS and not step.fixed_order and step.act_dtype == torch.bfloat16 and H % 4 == 0
        if add:
            y = step.buffer("block.sublayer_sum", (T, H), torch.float32)
            if not step.extra.get("block.sublayer_sum is clear"):
                ops.clear(y)
                step.extra["block.sublayer_sum is clear"] = True
        else:
            y = step.buffer("block.sublayer", (T, H), torch.float32)
        if step.act_dtype == torch.float32:
            x = h                           # (the sublayers read the 32-bit stream as it lies)
        else:
            x = step.buffer("block.stream_copy", (T, H), step.act_dtype)
            if step.extra.pop("block.stream_copy is for", None) != id(self):
                ops.copy_cols(h, x)
        self.mixer.forward(x, step, cache, y, add, write_cache)
        hand_on = isinstance(self.next_block, OutputNormBlock) and x is not h
        c, scales = self.residual_scale, self.scales or [None, None]
        # (the last sum into the stream leaves the copy of the rows only where the block behind reads it)
        last = 2 if self.token_input is not None else 1 if self.feed_forward is not None else 0
        self._join(y, self.mixer_norm, h, x if hand_on or last > 0 else h, add, c, scales[0])
        if self.feed_forward is not None:
            copy = x if hand_on or last > 1 else h
            rms = self.ffn_norm.fused_rms()
            if rms is not None and self.feed_forward.fuses_output_norm(h, step):
                self.feed_forward.forward_normed(x, step, h, scales[1] if scales[1] is not None else rms[0], rms[1], c,
                                                 copy if copy is not h else None)
            else:
                self.feed_forward.forward(x, step, y, add)
                self._join(y, self.ffn_norm, h, copy, add, c, scales[1])
        if self.token_input is not None:
            self.token_input.forward(x, step, y, add)
            self._join(y, self.token_input.norm, h, x if hand_on else h, add)
        if hand_on:
            step.extra["block.stream_copy is for"] = id(self.next_block)


register_part("block", "prenorm", PreNormBlock)
register_part("block", "output_norm", OutputNormBlock)
register_part("block", "parallel", ParallelBlock)
register_part("block", "sandwich", SandwichBlock)
