"""Typed configuration of the Salolorn decoder, read from config.json's own keys.

A Salolorn model is a list of layers whose branches each stand between two RMS norms, ``x += norm1b(mixer(norm1(x)))``, then ``x +=
norm2b(ff(norm2(x)))``; a stretch of the layers may run several times in a row with the same weights, each pass with caches and
states of its own, a learned vector ahead of each pass and the embedding's output again ahead of each but the first.  The mixer is
``latent_attention`` (one normed latent and one rotated key part a token for all heads, neighbouring pairs rotated, every earlier
token seen), ``delta`` (the gated delta rule behind short convolutions) or ``parallel``: grouped-query attention over chunks of
positions (a norm per head on q and k, half rotated against half, a sink and a sigmoid gate per head) beside gated linear attention
(a decay per key channel), both reading the same input, each times a factor.  The feed-forward is dense and gated (SiLU), or absent.
The head is the embedding table, its logits scaled.

Keys: ``architecture``, ``vocab``, ``width``, ``norm.eps``, ``logit_scale``, ``loop`` (``{"start", "stop", "times"}``; absent: every layer runs
once), and ``layers``, a list of ``{"type", "mixer": {...}, "mlp": {"kind": "dense", "ff"} | null}``.  Every size and constant comes from
there, but for the bottleneck of the linear attention's decays, which is that of its tensors; a missing or ill-typed key is an
error that names it.  Tensor names: ``embed``, ``loop.step``, ``final.norm``, and per layer ``l<i>.norm1 | norm1b | norm2 | norm2b``,
``l<i>.mix.*`` (``l<i>.mix.left.*`` and ``l<i>.mix.right.*`` side by side) and ``l<i>.mlp.gate | up | down``.
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Optional, Tuple

from .renanex import _get, _int, _num
from .specs import (ChunkedAttentionSpec, ConfigError, EmbeddingSpec, GatedDeltaSpec, GatedLinearSpec, GatedMlpSpec, HeadSpec,
                    LatentAttentionSpec, LoopStepsSpec, ModelSpec, NormSpec, RotarySpec, SandwichLayerSpec, SideBySideSpec)

ARCHITECTURE = "Salolorn"
# the configuration names no longest sequence: positions are 32-bit integers, and the pools bound a request
MAX_POSITIONS = 1 << 30
# the rank of the decays' bottleneck in a random checkpoint: config.json does not name it, a checkpoint's tensors have their own
RANDOM_DECAY_RANK = 16


@dataclass(frozen=True)
class LatentLayer:
    heads: int
    dim: int
    rot_dim: int
    vdim: int
    kv_rank: int
    scale: float
    base: float
    type: str = "latent_attention"


@dataclass(frozen=True)
class DeltaLayer:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    conv: int
    type: str = "delta"


@dataclass(frozen=True)
class ChunkedBranch:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    base: float
    rot_dims: int
    chunk: int


@dataclass(frozen=True)
class LinearBranch:
    heads: int
    dim: int
    vdim: int
    tau: float


@dataclass(frozen=True)
class ParallelLayer:
    left: ChunkedBranch
    right: LinearBranch
    left_scale: float
    right_scale: float
    type: str = "parallel"


def _grouped(m: dict, where: str) -> Tuple[int, int]:
    heads, kv = _int(m, "heads", where), _int(m, "kv_heads", where)
    if heads % kv:
        raise ConfigError(f"config.json: '{where}heads' {heads} is not a multiple of '{where}kv_heads' {kv}")
    return heads, kv


def _rot_of(m: dict, where: str, most: int) -> Tuple[float, int]:
    r, where = _get(m, "rot", where), where + "rot."
    dims = _int(r, "dims", where, 2)
    if dims % 2 or dims > most:
        raise ConfigError(f"config.json: '{where}dims' {dims} must be even and at most {most}")
    return _num(r, "base", where), dims


def _mixer_of(kind, m: dict, where: str):
    if kind == "latent_attention":
        rot_dim = _int(m, "rot_dim", where, 2)
        base, dims = _rot_of(m, where, rot_dim)
        if dims != rot_dim:
            raise ConfigError(f"config.json: '{where}rot.dims' must equal '{where}rot_dim' {rot_dim}: the whole part is rotated")
        return LatentLayer(_int(m, "heads", where), _int(m, "dim", where), rot_dim, _int(m, "vdim", where), _int(m, "kv_rank", where),
                           _num(m, "scale", where), base)
    if kind == "delta":
        heads, kv = _grouped(m, where)
        return DeltaLayer(heads, kv, _int(m, "dim", where), _int(m, "vdim", where), _int(m, "conv", where))
    if kind == "parallel":
        left, right = _get(m, "left", where), _get(m, "right", where)
        lw, rw = where + "left.", where + "right."
        heads, kv = _grouped(left, lw)
        dim = _int(left, "dim", lw)
        base, dims = _rot_of(left, lw, dim)
        return ParallelLayer(ChunkedBranch(heads, kv, dim, _int(left, "vdim", lw), _num(left, "scale", lw), base, dims,
                                           _int(_get(left, "mask", lw), "size", lw + "mask.")),
                             LinearBranch(_int(right, "heads", rw), _int(right, "dim", rw), _int(right, "vdim", rw), _num(right, "tau", rw)),
                             _num(m, "left_scale", where, positive=False), _num(m, "right_scale", where, positive=False))
    raise ConfigError(f"config.json: '{where[:-6]}type' {kind!r} is not a mixer of this architecture (delta, latent_attention, parallel)")


def _mlp_of(mlp, where: str) -> Optional[int]:
    if mlp is None:
        return None
    if not isinstance(mlp, dict):
        raise ConfigError(f"config.json: '{where[:-1]}' must be an object or null")
    kind = _get(mlp, "kind", where)
    if kind != "dense":
        raise ConfigError(f"config.json: '{where}kind' {kind!r} is not a feed-forward of this architecture (dense)")
    return _int(mlp, "ff", where)


def _loop_of(raw: dict, n: int) -> Optional[Tuple[int, int, int]]:
    if raw.get("loop") is None:
        return None
    loop = raw["loop"]
    start, stop, times = _int(loop, "start", "loop.", 0), _int(loop, "stop", "loop."), _int(loop, "times", "loop.")
    if not start < stop <= n:
        raise ConfigError(f"config.json: 'loop.start' {start} and 'loop.stop' {stop} must enclose layers of the {n}")
    return start, stop, times


@dataclass(frozen=True)
class SalolornConfig:
    vocab: int
    width: int
    norm_eps: float
    logit_scale: float
    loop: Optional[Tuple[int, int, int]]  # start, stop, times
    mixers: tuple
    ff: tuple                             # per layer the feed-forward's size, or None

    @classmethod
    def from_dict(cls, raw: dict) -> "SalolornConfig":
        layers = _get(raw, "layers", "")
        if not isinstance(layers, list) or not layers:
            raise ConfigError("config.json: 'layers' must be a list of at least one layer")
        mixers, ff = [], []
        for i, layer in enumerate(layers):
            where = f"layers[{i}]."
            if not isinstance(layer, dict):
                raise ConfigError(f"config.json: 'layers[{i}]' must be an object")
            mixers.append(_mixer_of(_get(layer, "type", where), _get(layer, "mixer", where), where + "mixer."))
            ff.append(_mlp_of(layer.get("mlp"), where + "mlp."))
        return cls(vocab=_int(raw, "vocab", ""), width=_int(raw, "width", ""), norm_eps=_num(_get(raw, "norm", ""), "eps", "norm."),
                   logit_scale=_num(raw, "logit_scale", "", positive=False), loop=_loop_of(raw, len(layers)), mixers=tuple(mixers), ff=tuple(ff))

    # ------------------------------------------------------------------ back to config.json
    def to_dict(self) -> dict:
        layers = []
        for m, ff in zip(self.mixers, self.ff):
            if isinstance(m, LatentLayer):
                mixer = {"heads": m.heads, "dim": m.dim, "rot_dim": m.rot_dim, "vdim": m.vdim, "kv_rank": m.kv_rank, "scale": m.scale,
                         "rot": {"base": m.base, "dims": m.rot_dim}}
            elif isinstance(m, DeltaLayer):
                mixer = {"heads": m.heads, "kv_heads": m.kv_heads, "dim": m.dim, "vdim": m.vdim, "conv": m.conv}
            else:
                a, b = m.left, m.right
                mixer = {"left": {"heads": a.heads, "kv_heads": a.kv_heads, "dim": a.dim, "vdim": a.vdim, "scale": a.scale,
                                  "rot": {"base": a.base, "dims": a.rot_dims}, "mask": {"size": a.chunk}},
                         "right": {"heads": b.heads, "dim": b.dim, "vdim": b.vdim, "tau": b.tau},
                         "left_scale": m.left_scale, "right_scale": m.right_scale}
            layers.append({"type": m.type, "mixer": mixer, "mlp": None if ff is None else {"kind": "dense", "ff": ff}})
        out = {"architecture": ARCHITECTURE, "vocab": self.vocab, "width": self.width, "norm": {"eps": self.norm_eps},
               "logit_scale": self.logit_scale, "layers": layers}
        if self.loop is not None:
            out["loop"] = dict(zip(("start", "stop", "times"), self.loop))
        return out

    # ------------------------------------------------------------------ the model as data
    def _mixer_spec(self, m, p: str):
        names = lambda q, *tensors: {(f"{s}.weight" if "." not in s and s not in ("sink", "norm", "A_log", "dt_bias") else s): q + s for s in tensors}
        if isinstance(m, LatentLayer):
            rotary = RotarySpec("rotary", m.rot_dim, m.base, table_precision="float64", pairing="neighbours")
            return LatentAttentionSpec("latent_attention", self.width, m.heads, m.dim, m.rot_dim, m.vdim, 0, m.kv_rank, m.scale, rotary,
                                       self.norm_eps, tensors=names(p, "q", "dkv", "dkv.norm", "uk", "uv", "o"))
        if isinstance(m, DeltaLayer):
            return GatedDeltaSpec("gated_delta", self.width, m.heads, m.kv_heads, m.dim, m.vdim, m.conv, self.norm_eps,
                                  names(p, "q", "q.conv", "k", "k.conv", "v", "v.conv", "g", "b", "a", "A_log", "dt_bias", "norm", "o"))
        a, b = m.left, m.right
        rotary = RotarySpec("rotary", a.dim, a.base, rotary_dim=a.rot_dims, table_precision="float64", pairing="halves")
        left = ChunkedAttentionSpec("chunked_attention", self.width, a.heads, a.kv_heads, a.dim, a.vdim, a.scale, rotary, bias=False, qk_norm=False,
                                    norm_eps=self.norm_eps, chunk=a.chunk, head_norm=True, sink=True, head_gate=True,
                                    tensors=names(p + "left.", "q", "q.norm", "k", "k.norm", "v", "g", "sink", "o"))
        right = GatedLinearSpec("gated_linear", self.width, b.heads, b.dim, b.vdim, b.tau, None, self.norm_eps,
                                dict(names(p + "right.", "q", "k", "v", "g", "a1", "a2", "norm", "o"), **{"a2.bias": p + "right.a2.b"}))
        return SideBySideSpec("side_by_side", self.width, (left, right), self.norm_eps, factors=(m.left_scale, m.right_scale))

    def _norm(self, name: str, ignored=()) -> NormSpec:
        return NormSpec("rmsnorm", self.width, self.norm_eps, {"weight": name}, ignored=tuple(ignored))

    def to_spec(self) -> ModelSpec:
        layers = []
        for i, (m, ff) in enumerate(zip(self.mixers, self.ff)):
            feed = norm2 = norm2b = None
            # a layer without feed-forward does not use its second norms, should the checkpoint have them
            unused = (f"l{i}.norm2", f"l{i}.norm2b") if ff is None else ()
            if ff is not None:
                feed = GatedMlpSpec("gated_mlp", self.width, ff, "silu", {f"{s}.weight": f"l{i}.mlp.{s}" for s in ("gate", "up", "down")},
                                    fill=True)
                norm2, norm2b = self._norm(f"l{i}.norm2"), self._norm(f"l{i}.norm2b")
            layers.append(SandwichLayerSpec("sandwich", self._mixer_spec(m, f"l{i}.mix."), feed, self._norm(f"l{i}.norm1", unused),
                                            self._norm(f"l{i}.norm1b"), norm2, norm2b))
        n, order, steps = len(layers), tuple(range(len(layers))), None
        if self.loop is not None:
            start, stop, times = self.loop
            order = tuple(range(start)) + tuple(range(start, stop)) * times + tuple(range(stop, n))
            steps = LoopStepsSpec(self.width, tuple(start + t * (stop - start) for t in range(times)), {"step": "loop.step"})
        spec = ModelSpec(architecture=ARCHITECTURE, embedding=EmbeddingSpec(self.vocab, self.width, {"weight": "embed"}), layers=tuple(layers),
                         order=order, final_norm=self._norm("final.norm"), head=HeadSpec(self.vocab, self.width, True, scale=self.logit_scale),
                         max_positions=MAX_POSITIONS, loop_steps=steps)
        spec.validate()
        return spec

    # ------------------------------------------------------------------ random weights
    def random_tensor_plan(self):
        """(name, shape, law) of every tensor of a random checkpoint; the laws are those of ``weights.random_init``."""
        w = self.width
        plan = [("embed", (self.vocab, w), "matrix")]
        if self.loop is not None:
            plan.append(("loop.step", (self.loop[2], w), "matrix"))
        for i, (m, ff) in enumerate(zip(self.mixers, self.ff)):
            p, q = f"l{i}.mix.", f"l{i}.mlp."
            plan += [(f"l{i}.{s}", (w,), "norm") for s in (("norm1", "norm1b") if ff is None else ("norm1", "norm1b", "norm2", "norm2b"))]
            if isinstance(m, LatentLayer):
                plan += [(p + "q", (m.heads * (m.dim + m.rot_dim), w), "matrix"), (p + "dkv", (m.kv_rank + m.rot_dim, w), "matrix"),
                         (p + "dkv.norm", (m.kv_rank,), "norm"), (p + "uk", (m.heads * m.dim, m.kv_rank), "matrix"),
                         (p + "uv", (m.heads * m.vdim, m.kv_rank), "matrix"), (p + "o", (w, m.heads * m.vdim), "matrix")]
            elif isinstance(m, DeltaLayer):
                for s, n in (("q", m.kv_heads * m.dim), ("k", m.kv_heads * m.dim), ("v", m.heads * m.vdim)):
                    plan += [(p + s, (n, w), "matrix"), (p + s + ".conv", (n, m.conv), "filter")]
                plan += [(p + "b", (m.heads, w), "matrix"), (p + "A_log", (m.heads,), "a_log"), (p + "norm", (m.vdim,), "norm"),
                         (p + "a", (m.heads, w), "matrix"), (p + "dt_bias", (m.heads,), "step_bias"), (p + "g", (m.heads * m.vdim, w), "matrix"),
                         (p + "o", (w, m.heads * m.vdim), "matrix")]
            else:
                a, b = m.left, m.right
                lp, rp, rank = p + "left.", p + "right.", RANDOM_DECAY_RANK
                plan += [(lp + "q", (a.heads * a.dim, w), "matrix"), (lp + "k", (a.kv_heads * a.dim, w), "matrix"), (lp + "v", (a.kv_heads * a.vdim, w), "matrix"),
                         (lp + "q.norm", (a.dim,), "norm"), (lp + "k.norm", (a.dim,), "norm"), (lp + "sink", (a.heads,), "filter"),
                         (lp + "g", (a.heads, w), "matrix"), (lp + "o", (w, a.heads * a.vdim), "matrix"),
                         (rp + "q", (b.heads * b.dim, w), "matrix"), (rp + "k", (b.heads * b.dim, w), "matrix"), (rp + "v", (b.heads * b.vdim, w), "matrix"),
                         (rp + "g", (b.heads * b.vdim, w), "matrix"), (rp + "o", (w, b.heads * b.vdim), "matrix"), (rp + "norm", (b.vdim,), "norm"),
                         (rp + "a1", (rank, w), "matrix"), (rp + "a2", (b.heads * b.dim, rank), "filter"), (rp + "a2.b", (b.heads * b.dim,), "bias")]
            if ff is not None:
                plan += [(q + "gate", (ff, w), "matrix"), (q + "up", (ff, w), "matrix"), (q + "down", (w, ff), "matrix")]
        return plan + [("final.norm", (w,), "norm")]
