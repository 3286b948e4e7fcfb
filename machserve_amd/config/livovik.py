"""Typed configuration of the Livovik decoder, read from config.json's own keys.

A Livovik model is a list of layers whose norms come after the sums: ``x <- norm1(alpha x + mixer(x))``, then ``x <-
norm2(alpha x + ff(x))``, RMS norms with plain weights and ``alpha`` one number for the model; the branches read ``x`` itself.
The mixer is ``attention``: grouped-query attention over chunks of positions with values of a width of their own, an RMS
norm per head on q and k, a rotation of half against half on part of a head with frequencies scaled by wavelength, a sink
and a sigmoid gate per head.  The feed-forward is ``dense`` (two products around the square of relu), ``moe`` (gated experts
with SiLU whose inputs are multiplied by the sigmoid scores of the chosen ones, and an expert for every token behind a
sigmoid gate of its own), or absent.  A layer with ``weights_of`` runs another layer's parts again with a cache of its own.

Keys: ``architecture``, ``vocab``, ``width``, ``norm.eps``, ``postln_alpha``, and ``layers``, a list of ``{"type", "mixer":
{...}, "mlp": {"kind": "dense", "ff"} | {"kind": "moe", "expert": {"ff"}, "router": {"experts", "top"}, "shared": {"ff"}} |
null, "weights_of"}``.  Every size and constant comes from there; a missing or ill-typed key is an error that names it.
Tensor names: ``embed``, ``head``, ``final.norm``, and per layer ``l<i>.norm1 | norm2``, ``l<i>.mix.*`` and ``l<i>.mlp.*``.
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Optional, Tuple

from .renanex import _get, _int, _num
from .specs import (ChunkedAttentionSpec, ConfigError, EmbeddingSpec, HeadSpec, ModelSpec, NormSpec, PlainMlpSpec, RotarySpec,
                    RoutedMlpSpec, SumNormLayerSpec, WavelengthScalingSpec)

ARCHITECTURE = "Livovik"
# the configuration names no longest sequence: positions are 32-bit integers, and the pools bound a request
MAX_POSITIONS = 1 << 30


@dataclass(frozen=True)
class Rotation:
    base: float
    dims: int
    scaling: Optional[Tuple[float, float, float, float]]  # factor, low, high, original; None: frequencies as they are


@dataclass(frozen=True)
class AttentionLayer:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    rot: Optional[Rotation]
    chunk: Optional[int]  # None: plain causal
    type: str = "attention"


@dataclass(frozen=True)
class DenseMlp:
    ff: int
    kind: str = "dense"


@dataclass(frozen=True)
class ExpertsMlp:
    experts: int
    top: int
    ff: int
    shared: int  # 0: no expert that every token uses
    kind: str = "moe"


def _rotation_of(m: dict, where: str, dim: int) -> Optional[Rotation]:
    if m.get("rot") is None:
        return None
    r, where = m["rot"], where + "rot."
    dims = _int(r, "dims", where, 2)
    if dims % 2 or dims > dim:
        raise ConfigError(f"config.json: '{where}dims' {dims} must be even and at most the head size {dim}")
    scaling = None
    if r.get("scaling") is not None:
        scaling = tuple(_num(r["scaling"], k, where + "scaling.") for k in ("factor", "low", "high", "original"))
        if scaling[1] > scaling[2]:
            raise ConfigError(f"config.json: '{where}scaling.low' {scaling[1]} exceeds '{where}scaling.high' {scaling[2]}")
    return Rotation(_num(r, "base", where), dims, scaling)


def _mixer_of(kind, m: dict, where: str) -> AttentionLayer:
    if kind != "attention":
        raise ConfigError(f"config.json: '{where[:-6]}type' {kind!r} is not a mixer of this architecture (attention)")
    heads, kv = _int(m, "heads", where), _int(m, "kv_heads", where)
    if heads % kv:
        raise ConfigError(f"config.json: '{where}heads' {heads} is not a multiple of '{where}kv_heads' {kv}")
    dim = _int(m, "dim", where)
    chunk = _int(m["mask"], "size", where + "mask.") if m.get("mask") is not None else None
    return AttentionLayer(heads, kv, dim, _int(m, "vdim", where), _num(m, "scale", where), _rotation_of(m, where, dim), chunk)


def _mlp_of(mlp, where: str):
    if mlp is None:
        return None
    if not isinstance(mlp, dict):
        raise ConfigError(f"config.json: '{where[:-1]}' must be an object or null")
    kind = _get(mlp, "kind", where)
    if kind == "dense":
        return DenseMlp(_int(mlp, "ff", where))
    if kind == "moe":
        router = _get(mlp, "router", where)
        experts, top = _int(router, "experts", where + "router."), _int(router, "top", where + "router.")
        if top > experts:
            raise ConfigError(f"config.json: '{where}router.top' {top} exceeds '{where}router.experts' {experts}")
        shared = mlp.get("shared")
        return ExpertsMlp(experts, top, _int(_get(mlp, "expert", where), "ff", where + "expert."),
                          _int(shared, "ff", where + "shared.") if shared is not None else 0)
    raise ConfigError(f"config.json: '{where}kind' {kind!r} is not a feed-forward of this architecture (dense, moe)")


def _owners(sources) -> tuple:
    """For every layer the layer whose tensors it uses: itself, or what its ``weights_of`` leads to."""
    owners = []
    for i, src in enumerate(sources):
        where, seen = f"layers[{i}].weights_of", {i}
        at = i
        while sources[at] is not None:
            at = sources[at]
            if isinstance(at, bool) or not isinstance(at, int) or not 0 <= at < len(sources):
                raise ConfigError(f"config.json: '{where}' must name a layer, got {at!r}")
            if at in seen:
                raise ConfigError(f"config.json: '{where}' leads back to layer {at}: no layer has tensors of its own")
            seen.add(at)
        owners.append(at)
    return tuple(owners)


@dataclass(frozen=True)
class LivovikConfig:
    vocab: int
    width: int
    norm_eps: float
    alpha: float
    mixers: tuple
    mlps: tuple
    owners: tuple  # layer -> the layer whose tensors it uses

    @classmethod
    def from_dict(cls, raw: dict) -> "LivovikConfig":
        layers = _get(raw, "layers", "")
        if not isinstance(layers, list) or not layers:
            raise ConfigError("config.json: 'layers' must be a list of at least one layer")
        mixers, mlps, sources = [], [], []
        for i, layer in enumerate(layers):
            where = f"layers[{i}]."
            if not isinstance(layer, dict):
                raise ConfigError(f"config.json: 'layers[{i}]' must be an object")
            mixers.append(_mixer_of(_get(layer, "type", where), _get(layer, "mixer", where), where + "mixer."))
            mlps.append(_mlp_of(layer.get("mlp"), where + "mlp."))
            sources.append(layer.get("weights_of"))
        owners = _owners(sources)
        for i, j in enumerate(owners):
            if (mixers[i], mlps[i]) != (mixers[j], mlps[j]):
                raise ConfigError(f"config.json: 'layers[{i}]' uses the weights of layer {j}, but their mixers or feed-forwards differ")
        return cls(vocab=_int(raw, "vocab", ""), width=_int(raw, "width", ""), norm_eps=_num(_get(raw, "norm", ""), "eps", "norm."),
                   alpha=_num(raw, "postln_alpha", "", positive=False), mixers=tuple(mixers), mlps=tuple(mlps), owners=owners)

    # ------------------------------------------------------------------ back to config.json
    def to_dict(self) -> dict:
        layers = []
        for i, (m, mlp) in enumerate(zip(self.mixers, self.mlps)):
            mixer = {"heads": m.heads, "kv_heads": m.kv_heads, "dim": m.dim, "vdim": m.vdim, "scale": m.scale}
            if m.rot is not None:
                mixer["rot"] = {"base": m.rot.base, "dims": m.rot.dims}
                if m.rot.scaling is not None:
                    mixer["rot"]["scaling"] = dict(zip(("factor", "low", "high", "original"), m.rot.scaling))
            if m.chunk is not None:
                mixer["mask"] = {"size": m.chunk}
            ff = None
            if isinstance(mlp, DenseMlp):
                ff = {"kind": "dense", "ff": mlp.ff}
            elif isinstance(mlp, ExpertsMlp):
                ff = {"kind": "moe", "expert": {"ff": mlp.ff}, "router": {"experts": mlp.experts, "top": mlp.top}}
                if mlp.shared:
                    ff["shared"] = {"ff": mlp.shared}
            layer = {"type": m.type, "mixer": mixer, "mlp": ff}
            if self.owners[i] != i:
                layer["weights_of"] = self.owners[i]
            layers.append(layer)
        return {"architecture": ARCHITECTURE, "vocab": self.vocab, "width": self.width, "norm": {"eps": self.norm_eps},
                "postln_alpha": self.alpha, "layers": layers}

    # ------------------------------------------------------------------ the model as data
    def _mixer_spec(self, m: AttentionLayer, p: str) -> ChunkedAttentionSpec:
        rotary = None
        if m.rot is not None:
            bands = WavelengthScalingSpec(*m.rot.scaling) if m.rot.scaling is not None else None
            rotary = RotarySpec("rotary", m.dim, m.rot.base, rotary_dim=m.rot.dims, table_precision="float64", pairing="halves",
                                wavelengths=bands)
        names = {f"{s}.weight": p + s for s in ("q", "k", "v", "g", "o")}
        names.update({"q.norm": p + "q.norm", "k.norm": p + "k.norm", "sink": p + "sink"})
        return ChunkedAttentionSpec("chunked_attention", self.width, m.heads, m.kv_heads, m.dim, m.vdim, m.scale, rotary, bias=False,
                                    qk_norm=False, norm_eps=self.norm_eps, chunk=m.chunk, tensors=names, head_norm=True, sink=True,
                                    head_gate=True)

    def _mlp_spec(self, mlp, q: str):
        if isinstance(mlp, DenseMlp):
            return PlainMlpSpec("plain_mlp", self.width, mlp.ff, "relu2", {"up.weight": q + "up", "down.weight": q + "down"})
        names = {"router.weight": q + "router", "shared.gate_weight": q + "shared.sg"}
        for e in [f"e{i}" for i in range(mlp.experts)] + ["shared"]:
            names.update({f"{e}.{s}": q + f"{e}.{s}" for s in ("gate", "up", "down")})
        return RoutedMlpSpec("routed_mlp", self.width, mlp.experts, mlp.top, mlp.ff, "silu", mlp.shared, False, names, gated=True,
                             scoring="sigmoid", weigh="input", shared_gate=mlp.shared > 0)

    def _norm(self, name: str, ignored=()) -> NormSpec:
        return NormSpec("rmsnorm", self.width, self.norm_eps, {"weight": name}, ignored=tuple(ignored))

    def to_spec(self) -> ModelSpec:
        layers, built = [], {}
        for i, (m, mlp) in enumerate(zip(self.mixers, self.mlps)):
            if self.owners[i] != i:
                continue
            built[i] = len(layers)
            # a layer without feed-forward does not use its second norm, should the checkpoint have it
            norm1 = self._norm(f"l{i}.norm1", () if mlp is not None else (f"l{i}.norm2",))
            layers.append(SumNormLayerSpec("sumnorm", self._mixer_spec(m, f"l{i}.mix."),
                                           self._mlp_spec(mlp, f"l{i}.mlp.") if mlp is not None else None, norm1,
                                           self._norm(f"l{i}.norm2") if mlp is not None else None, self.alpha))
        spec = ModelSpec(architecture=ARCHITECTURE, embedding=EmbeddingSpec(self.vocab, self.width, {"weight": "embed"}),
                         layers=tuple(layers), order=tuple(built[j] for j in self.owners), final_norm=self._norm("final.norm"),
                         head=HeadSpec(self.vocab, self.width, False, {"weight": "head"}), max_positions=MAX_POSITIONS)
        spec.validate()
        return spec

    # ------------------------------------------------------------------ random weights
    def random_tensor_plan(self):
        """(name, shape, law) of every tensor of a random checkpoint; the laws are those of ``weights.random_init``."""
        w = self.width
        plan = [("embed", (self.vocab, w), "matrix")]
        for i, (m, mlp) in enumerate(zip(self.mixers, self.mlps)):
            if self.owners[i] != i:
                continue
            p, q = f"l{i}.mix.", f"l{i}.mlp."
            plan += [(f"l{i}.norm1", (w,), "norm")] + ([(f"l{i}.norm2", (w,), "norm")] if mlp is not None else [])
            plan += [(p + "q", (m.heads * m.dim, w), "matrix"), (p + "k", (m.kv_heads * m.dim, w), "matrix"),
                     (p + "v", (m.kv_heads * m.vdim, w), "matrix"), (p + "q.norm", (m.dim,), "norm"), (p + "k.norm", (m.dim,), "norm"),
                     (p + "sink", (m.heads,), "filter"), (p + "g", (m.heads, w), "matrix"), (p + "o", (w, m.heads * m.vdim), "matrix")]
            if isinstance(mlp, DenseMlp):
                plan += [(q + "up", (mlp.ff, w), "matrix"), (q + "down", (w, mlp.ff), "matrix")]
            elif isinstance(mlp, ExpertsMlp):
                experts = [(f"e{e}", mlp.ff) for e in range(mlp.experts)] + ([("shared", mlp.shared)] if mlp.shared else [])
                for e, ff in experts:
                    plan += [(q + f"{e}.gate", (ff, w), "matrix"), (q + f"{e}.up", (ff, w), "matrix"), (q + f"{e}.down", (w, ff), "matrix")]
                plan.append((q + "router", (mlp.experts, w), "filter"))
                if mlp.shared:
                    plan.append((q + "shared.sg", (1, w), "filter"))
        return plan + [("final.norm", (w,), "norm"), ("head", (self.vocab, w), "matrix")]
