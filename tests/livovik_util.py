"""Small Livovik configurations, model folders made from them and the plain model's logits."""
from __future__ import annotations

import json
import os

import torch

from plain import livovik_plain as P
from renanex_util import relative_error, relative_errors, run_schedule, tokens_of  # noqa: F401  (shared runners)


def attention(heads, kv, dim, vdim, scale, chunk=16, rot=(10000.0, None), scaling=None):
    m = {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "scale": scale}
    if rot is not None:
        m["rot"] = {"base": rot[0], "dims": rot[1] or dim}
        if scaling is not None:
            m["rot"]["scaling"] = dict(zip(("factor", "low", "high", "original"), scaling))
    if chunk:
        m["mask"] = {"size": chunk}
    return m


def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(experts, top, ff, shared=None):
    m = {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}
    if shared:
        m["shared"] = {"ff": shared}
    return m


def layer(mixer, mlp):
    return {"type": "attention", "mixer": mixer, "mlp": mlp}


def model(width, vocab, layers, alpha, eps=1e-6):
    """A layer given as a number runs that layer's tensors again."""
    entries = [dict(layers[e], weights_of=e) if isinstance(e, int) else e for e in layers]
    return {"architecture": "Livovik", "vocab": vocab, "width": width, "norm": {"eps": eps}, "postln_alpha": alpha, "layers": entries}


CONFIGS = {
    # two of the layers run again; values wider and narrower than keys; a rotation of part of a head with scaled
    # frequencies, of the whole head without scaling, and none; chunks that are and are not a multiple of a page of 16, and
    # none; experts with and without one for every token; a layer without feed-forward
    "mixed": model(64, 97, [
        layer(attention(4, 2, 16, 24, 0.3, 16, (500.0, 8), (4.0, 1.0, 3.0, 64)), moe(6, 2, 24, shared=40)),
        layer(attention(4, 1, 24, 16, 0.2, 24, (10000.0, 24)), dense(80)),
        0,
        layer(attention(2, 2, 16, 16, 0.35, None, None), moe(5, 3, 16)),
        1,
        layer(attention(3, 3, 32, 8, 0.15, 20, (100.0, 16), (8.0, 0.5, 8.0, 40)), None)], alpha=1.7),
    # sizes that are no multiples of 8 or 16, a chunk shorter than a page, one key/value head under six heads, one expert a
    # token, every expert a token, a layer that runs the tensors of a later one and one that does so through it
    "odd": {"architecture": "Livovik", "vocab": 61, "width": 48, "norm": {"eps": 1e-5}, "postln_alpha": 0.9, "layers": [
        dict(layer(attention(6, 1, 20, 12, 0.3, 7, (100.0, 6), (3.0, 1.0, 1.0, 30)), moe(7, 1, 20, shared=12)), weights_of=2),
        layer(attention(2, 2, 10, 18, 0.5, 33, (1000.0, 10), (2.0, 0.25, 4.0, 12.5)), dense(36)),
        layer(attention(6, 1, 20, 12, 0.3, 7, (100.0, 6), (3.0, 1.0, 1.0, 30)), moe(7, 1, 20, shared=12)),
        layer(attention(3, 1, 8, 8, 0.6, 1, (50.0, 2)), moe(3, 3, 8, shared=8)),
        dict(layer(attention(6, 1, 20, 12, 0.3, 7, (100.0, 6), (3.0, 1.0, 1.0, 30)), moe(7, 1, 20, shared=12)), weights_of=0)]},
    # heads of 64 (the attention kernels' tile of 64 takes work items of another size in the two-byte types), a chunk
    # longer than the prompts of most tests, seventeen heads over one key/value head (beyond a decode tile), many experts
    "wide": model(128, 128, [
        layer(attention(4, 4, 64, 64, 0.12, 200, (250000.0, 32), (16.0, 1.0, 4.0, 128)), moe(32, 4, 32, shared=64)),
        layer(attention(17, 1, 16, 32, 0.3, 32, (1000.0, 16)), dense(256)),
        layer(attention(8, 2, 40, 64, 0.2, 100, (1000.0, 24)), moe(8, 8, 16))], alpha=2.5),
}

# configurations for the GPU alone (the stand-ins would take minutes): sizes nearer a real model's layers
MORE_CONFIGS = {
    "big": model(512, 1000, [
        layer(attention(8, 2, 128, 128, 0.088, 96, (500000.0, 64), (8.0, 1.0, 4.0, 256)), dense(1024)),
        layer(attention(8, 2, 64, 128, 0.125, 64, (10000.0, 64)), moe(16, 4, 128, shared=256)),
        1,
        layer(attention(8, 8, 128, 64, 0.088, 130, (10000.0, 32), (4.0, 1.0, 2.0, 100)), moe(8, 1, 256, shared=128)),
        0], alpha=2.2),
}
CONFIGS_ALL = dict(CONFIGS, **MORE_CONFIGS)


def make_dir(tmp, name: str, seed: int = 0, sharpen: float = 3.0, dtype=torch.float32, experts: float = 5.0) -> str:
    """A model folder of random weights, changed so that faults show: embeddings of order one, query norms times ``sharpen``
    (softmaxes far from flat: a key that is missing or one too many shows in the logits), sinks that take a good part
    of a softmax, and branches that weigh as much as the stream they are added to.  ``experts``: the factor on the routed
    experts' projections (large: a row whose choice flips under a two-byte type's rounding is lost)."""
    from safetensors.torch import load_file, save_file
    from machserve_amd.weights import write_random_model
    out = os.path.join(str(tmp), f"livovik_{name}_{seed}_{sharpen}_{experts}")
    write_random_model(dict(CONFIGS_ALL[name]), seed, out, dtype)
    path = os.path.join(out, "model.safetensors")
    w = load_file(path)
    for k in list(w):
        t = w[k].float()
        if k == "embed":
            t = t * 40.0
        elif k.endswith(".q.norm"):
            t = t * sharpen
        elif k.endswith(".sink"):
            t = t * 4.0 + 1.5
        elif ".mlp.e" in k:  # (projections: outputs of order one whatever they sum over)
            t = t * experts * (64.0 / t.shape[1]) ** 0.5
        elif k.endswith((".up", ".gate", ".down", ".mix.v", ".mix.o", ".mix.g", ".mix.q", ".mix.k")):
            t = t * 5.0 * (64.0 / t.shape[1]) ** 0.5
        elif k.endswith((".router", ".shared.sg")):
            t = t * (64.0 / t.shape[1]) ** 0.5
        w[k] = t.to(dtype)
    save_file(w, path)
    return out


def read(model_dir: str):
    from safetensors.torch import load_file
    with open(os.path.join(model_dir, "config.json")) as f:
        cfg = json.load(f)
    return load_file(os.path.join(model_dir, "model.safetensors")), cfg


def plain_logits(model_dir: str, tokens, dtype=torch.float64, weights_as=None) -> torch.Tensor:
    """The plain model's logits; ``weights_as``: matrices rounded to this type first, as a run in that type holds them."""
    w, cfg = read(model_dir)
    if weights_as is not None and weights_as != torch.float32:
        w = {k: v.to(weights_as).float() if _is_matrix(k, v) else v for k, v in w.items()}
    return P.forward(w, cfg, tokens, dtype)


def _is_matrix(name: str, t) -> bool:
    """What a run keeps in its element type: operands of matrix products and the embedding (not the router and its gate)."""
    return t.dim() == 2 and not name.endswith((".router", ".shared.sg"))


def within(got: torch.Tensor, want: torch.Tensor, dtype) -> bool:
    """float32: every row within rounding of sums taken in another order (a key too many or too few, a chunk one token off
    or a sink left out is off by 1e-2 and more).  bfloat16: rounding of activations grows through the layers, so half the
    rows must be within 4e-2; and where two router scores lie within that rounding of each other a row takes another
    expert than the plain model does, which moves that row by as much as the expert matters: at most one row in thirty
    may be beyond 0.25 (logits that have nothing to do with the wanted ones are off by 1.4 in every row)."""
    e = relative_errors(got, want)
    if dtype == torch.float32:
        return float(e.max()) < 1e-4
    return float(e.median()) < 4e-2 and int((e > 0.25).sum()) <= max(1, e.numel() // 30)
