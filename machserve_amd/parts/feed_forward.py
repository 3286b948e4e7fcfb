"""Dense gated feed-forward ``down(act(gate(x)) * up(x))``, activation on the gate branch
(``crates/mach-model/src/batched.rs:4424-4453``; SiLU: ``crates/mach-model/src/kernels.rs:131-140``,
the tanh form of GELU: ``crates/mach-model/src/kernels.rs:199-208``).  Which activation is the
specification's to say.  Gate and up are one product whose epilogue applies the activation; down
accumulates into the 32-bit stream.  With biases on every projection the gate/up product leaves 32-bit sums, a small kernel
adds the biases' effect (they ride in the product's epilogue), applies the activation and multiplies, and the down
projection's bias goes into the stream with its product.  Beside it the plain feed-forward without a gate branch,
``down(act(up(x)))``, whose activation is the up product's epilogue."""
from __future__ import annotations

import torch

from ..kernels.ops import GATE_ACTIVATIONS, UNARY_ACTIVATIONS, interleave_gate_up
from .base import FeedForward, PendingNorm, TensorDecl, require_kernel_sizes
from .registry import register_feed_forward


@register_feed_forward("gated_mlp")
class GatedMlp(FeedForward):
    takes_pending_norm = True  # its first product can apply the norm of the stream itself

    def __init__(self, spec, rt):
        super().__init__(spec, rt)
        if spec.activation not in GATE_ACTIVATIONS:
            raise ValueError(f"gated_mlp: activation {spec.activation!r} is not built (built: {', '.join(sorted(GATE_ACTIVATIONS))})")
        self.bias = bool(getattr(spec, "bias", False))
        # the joint size as the kernels see it: where the spec asks for it, filled up to a multiple of 8 by rows of zeros
        self.joint = -(-spec.intermediate // 8) * 8 if getattr(spec, "fill", False) and not self.bias else spec.intermediate
        require_kernel_sizes(rt, "gated_mlp", [("hidden size", spec.hidden), ("intermediate size", self.joint)])

    def tensor_decls(self):
        s = self.spec
        decls = [TensorDecl("gate.weight", (s.intermediate, s.hidden)), TensorDecl("up.weight", (s.intermediate, s.hidden)),
                 TensorDecl("down.weight", (s.hidden, s.intermediate))]
        if self.bias:
            decls += [TensorDecl("gate.bias", (s.intermediate,), "vector"), TensorDecl("up.bias", (s.intermediate,), "vector"),
                      TensorDecl("down.bias", (s.hidden,), "vector")]
        return decls

    def load(self, t):
        self.w_down = t["down.weight"]
        if self.bias:  # gate and up one after the other: their product leaves 32-bit sums that take the biases
            self.w_gate_up = torch.cat([t["gate.weight"], t["up.weight"]], dim=0).contiguous()
            self.b_gate_up = torch.cat([t["gate.bias"], t["up.bias"]]).contiguous()
            self.b_down = t["down.bias"]
        else:
            fill = self.joint - self.spec.intermediate
            pad = torch.nn.functional.pad
            self.w_gate_up = interleave_gate_up(pad(t["gate.weight"], (0, 0, 0, fill)), pad(t["up.weight"], (0, 0, 0, fill)))
            if fill:
                self.w_down = pad(self.w_down, (0, fill)).contiguous()

    def forward(self, h, stream, ctx):
        if self.bias:
            if isinstance(h, PendingNorm):
                h = h.tensor()
            sums = self.rt.ops.linear(h, self.w_gate_up, self.b_gate_up, out_f32=True)
            stream.add_linear(self.rt.ops.gate_mul(sums, self.spec.activation), self.w_down, self.b_down)
            return
        if isinstance(h, PendingNorm):
            a = h.linear_swiglu(self.w_gate_up, self.joint, self.spec.activation)
        else:
            a = self.rt.ops.linear_swiglu(h, self.w_gate_up, self.joint, self.spec.activation)
        stream.add_linear(a, self.w_down)


@register_feed_forward("plain_mlp")
class PlainMlp(FeedForward):
    """``down(act(up(x)))``; the joint size is filled up with zeros to a multiple of 8, which every activation built maps to zeros."""

    def __init__(self, spec, rt):
        super().__init__(spec, rt)
        if spec.activation not in UNARY_ACTIVATIONS:
            raise ValueError(f"plain_mlp: activation {spec.activation!r} is not built (built: {', '.join(sorted(UNARY_ACTIVATIONS))})")
        require_kernel_sizes(rt, "plain_mlp", [("hidden size", spec.hidden)])

    def tensor_decls(self):
        s = self.spec
        return [TensorDecl("up.weight", (s.intermediate, s.hidden)), TensorDecl("down.weight", (s.hidden, s.intermediate))]

    def load(self, t):
        fill = -self.spec.intermediate % 8
        pad = torch.nn.functional.pad
        self.w_up = pad(t["up.weight"], (0, 0, 0, fill)).contiguous()
        self.w_down = pad(t["down.weight"], (0, fill)).contiguous()

    def forward(self, h, stream, ctx):
        if isinstance(h, PendingNorm):
            h = h.tensor()
        stream.add_linear(self.rt.ops.linear_act(h, self.w_up, self.spec.activation), self.w_down)
