"""The gated delta rule as a mixer with state of fixed size: a write first takes away what the state holds for its key.

Per step: q, k, v, the output's gate, the step sizes and the decays' inputs as one product that leaves 32-bit sums; one kernel that
finishes a row (a causal convolution per channel of q, k and v with SiLU, whose last ``taps - 1`` inputs are state; unit vectors
per head of q and k; ``beta = sigmoid(b)``, ``g = exp(-exp(A_log) softplus(a + dt_bias))`` as its logarithm); the rule itself per
head, ``S <- g S``, ``u = beta (v - S^T k)``, ``S <- S + k u^T``, ``o = S^T q`` (decoded tokens in one pass over the state; portions in
chunks of 64 tokens as small matrix products, see ``ops.gated_delta``), with a head's root mean square divided out and the
weight and the gate's SiLU applied; the output projection.  Heads of q and k may be fewer than those of v: head h uses head
``h // (heads / kv_heads)``.  All of it but the two projections is 32-bit in every build.
"""
from __future__ import annotations

import torch

from .base import Mixer, StateRequest, TensorDecl, require_kernel_sizes
from .registry import register_mixer


@register_mixer("gated_delta")
class GatedDelta(Mixer):
    graph_safe = True  # reads the requests' rows and slots from device memory only

    def __init__(self, spec, rt):
        super().__init__(spec, rt)
        s = spec
        if s.heads % s.kv_heads:
            raise ValueError(f"gated_delta: {s.heads} heads are not a multiple of {s.kv_heads} query/key heads")
        self.nk, self.nv = s.kv_heads * s.head_dim, s.heads * s.v_head_dim
        self.channels = 2 * self.nk + self.nv
        self.out_cols = -(-self.nv // 8) * 8  # the output projection sums over a multiple of 8
        require_kernel_sizes(rt, "gated_delta", [("hidden size", s.hidden)])
        limits = getattr(rt.ops, "gated_state_limits", None)
        if limits is not None:
            lim = limits()
            if max(s.head_dim, s.v_head_dim) > lim["dim"] or not 1 <= s.conv_taps <= lim["taps"]:
                raise ValueError(f"gated_delta: heads of {s.head_dim} and {s.v_head_dim} under {s.conv_taps} taps; the kernels take up to "
                                 f"{lim['dim']} and 1 to {lim['taps']}")
        self.state = None

    def tensor_decls(self):
        s = self.spec
        decls = []
        for name, n in (("q", self.nk), ("k", self.nk), ("v", self.nv)):
            decls += [TensorDecl(f"{name}.weight", (n, s.hidden)), TensorDecl(f"{name}.conv", (n, s.conv_taps), "vector")]
        return decls + [TensorDecl("g.weight", (self.nv, s.hidden)), TensorDecl("b.weight", (s.heads, s.hidden)), TensorDecl("a.weight", (s.heads, s.hidden)),
                        TensorDecl("A_log", (s.heads,), "vector"), TensorDecl("dt_bias", (s.heads,), "vector"),
                        TensorDecl("norm", (s.v_head_dim,), "vector"), TensorDecl("o.weight", (s.hidden, self.nv))]

    def load(self, t):
        parts = [t[f"{n}.weight"] for n in ("q", "k", "v", "g", "b", "a")]
        fill = -sum(p.shape[0] for p in parts) % 8
        self.w_in = torch.cat(parts + ([parts[0].new_zeros((fill, self.spec.hidden))] if fill else []), dim=0).contiguous()
        self.conv_w = torch.cat([t[f"{n}.conv"] for n in ("q", "k", "v")], dim=0).contiguous()
        self.a_log, self.dt_bias, self.norm_w = t["A_log"], t["dt_bias"], t["norm"]
        self.w_o = torch.nn.functional.pad(t["o.weight"], (0, self.out_cols - self.nv)).contiguous()

    def cache_request(self):
        s = self.spec
        shapes = {"kv": (s.heads, s.head_dim, -(-s.v_head_dim // 4) * 4)}
        if s.conv_taps > 1:
            shapes["conv"] = (s.conv_taps - 1, self.channels)
        return StateRequest(shapes)

    def bind_cache(self, binding):
        self.state = binding.tensors

    def forward(self, h, stream, ctx):
        s, ops, single = self.spec, self.rt.ops, ctx.decode_only
        seqs, sizes = (ctx.seq_q_start, ctx.seq_q_len, ctx.seq_slot), (s.heads, s.kv_heads, s.head_dim, s.v_head_dim)
        sums = ops.linear_split(h, self.w_in)
        rows = ops.delta_rows(sums, self.conv_w, self.state.get("conv"), self.a_log, self.dt_bias, float(s.head_dim) ** -0.5, *seqs, *sizes, single=single)
        y = ops.gated_delta(*rows, sums, self.channels, self.norm_w, s.norm_eps, self.state["kv"], *seqs, *sizes, self.out_cols, single=single)
        stream.add_linear(y, self.w_o)
