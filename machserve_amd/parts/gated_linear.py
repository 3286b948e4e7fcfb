"""Gated linear attention as a mixer with state of fixed size: a decay per key channel that depends on the token.

Per step: q, k, v, the output's gate and the decay's bottleneck as one product that leaves 32-bit sums; the decays
``alpha = sigmoid(W_a2 low + b)^(1 / tau)``, worked out in 32-bit by one kernel; one kernel that carries the ``[dim, vdim]`` state of
every head (``S <- diag(alpha) S + k v^T``, ``o = S^T q``; decoded tokens in one pass over the state, long portions in segments side
by side, see ``ops.gated_linear``), divides a head's output by its root mean square and applies the weight and the gate's SiLU; the
output projection.  Decays, states and unit norms are 32-bit in every build.
"""
from __future__ import annotations

import torch

from .base import Mixer, StateRequest, TensorDecl, require_kernel_sizes
from .registry import register_mixer


@register_mixer("gated_linear")
class GatedLinearAttention(Mixer):
    graph_safe = True  # reads the requests' rows and slots from device memory only

    def __init__(self, spec, rt):
        super().__init__(spec, rt)
        s = spec
        self.nk, self.nv = s.heads * s.head_dim, s.heads * s.v_head_dim
        self.out_cols = -(-self.nv // 8) * 8  # the output projection sums over a multiple of 8
        require_kernel_sizes(rt, "gated_linear", [("hidden size", s.hidden)])
        limits = getattr(rt.ops, "gated_state_limits", None)
        if limits is not None and max(s.head_dim, s.v_head_dim) > limits()["dim"]:
            raise ValueError(f"gated_linear: heads of {s.head_dim} and {s.v_head_dim}; the kernels take up to {limits()['dim']}")
        self.state = None

    def tensor_decls(self):
        s, rank = self.spec, self.spec.decay_rank
        return [TensorDecl("q.weight", (self.nk, s.hidden)), TensorDecl("k.weight", (self.nk, s.hidden)), TensorDecl("v.weight", (self.nv, s.hidden)),
                TensorDecl("g.weight", (self.nv, s.hidden)), TensorDecl("a1.weight", (rank, s.hidden) if rank else None),
                TensorDecl("a2.weight", (self.nk, rank) if rank else None, "vector"), TensorDecl("a2.bias", (self.nk,), "vector"),
                TensorDecl("norm", (s.v_head_dim,), "vector"), TensorDecl("o.weight", (s.hidden, self.nv))]

    def load(self, t):
        s, a1, a2 = self.spec, t["a1.weight"], t["a2.weight"]
        if a1.shape[0] != a2.shape[1] or a1.shape[1] != s.hidden or a2.shape[0] != self.nk:
            raise ValueError(f"gated_linear: the decay's bottleneck {tuple(a1.shape)} and {tuple(a2.shape)} does not fit")
        limits = getattr(self.rt.ops, "gated_state_limits", None)
        if limits is not None and a1.shape[0] > limits()["rank"]:
            raise ValueError(f"gated_linear: a bottleneck of {a1.shape[0]}; the kernels take up to {limits()['rank']}")
        parts = [t["q.weight"], t["k.weight"], t["v.weight"], t["g.weight"], a1]
        fill = -sum(p.shape[0] for p in parts) % 8
        self.w_in = torch.cat(parts + ([a1.new_zeros((fill, s.hidden))] if fill else []), dim=0).contiguous()
        self.w_a2t, self.b_a2, self.norm_w = a2.t().contiguous(), t["a2.bias"], t["norm"]  # [rank, channels]: the kernel's threads are channels
        self.w_o = torch.nn.functional.pad(t["o.weight"], (0, self.out_cols - self.nv)).contiguous()

    def cache_request(self):
        s = self.spec
        return StateRequest({"kv": (s.heads, s.head_dim, -(-s.v_head_dim // 4) * 4)})

    def bind_cache(self, binding):
        self.state = binding.tensors

    def forward(self, h, stream, ctx):
        s, ops = self.spec, self.rt.ops
        sums = ops.linear_split(h, self.w_in)
        alpha = ops.key_decay(sums, 2 * self.nk + 2 * self.nv, self.w_a2t, self.b_a2, float(s.tau))
        y = ops.gated_linear(sums, alpha, self.norm_w, s.norm_eps, float(s.head_dim) ** -0.5, self.state["kv"], ctx.seq_q_start, ctx.seq_q_len,
                             ctx.seq_slot, s.heads, s.head_dim, s.v_head_dim, self.out_cols, single=ctx.decode_only)
        stream.add_linear(y, self.w_o)
