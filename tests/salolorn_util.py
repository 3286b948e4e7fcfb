"""Small Salolorn configurations, model folders made from them and the plain model's logits."""
from __future__ import annotations

import json
import os

import torch

from plain import salolorn_plain as P
from renanex_util import relative_error, relative_errors, run_schedule, tokens_of  # noqa: F401  (shared runners)


def latent(heads, dim, rot_dim, vdim, kv_rank, scale, base=10000.0):
    return {"type": "latent_attention", "mixer": {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank, "scale": scale,
                                                  "rot": {"base": base, "dims": rot_dim}}}


def delta(heads, kv, dim, vdim, conv):
    return {"type": "delta", "mixer": {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "conv": conv}}


def parallel(left, right, left_scale, right_scale):
    """left: (heads, kv_heads, dim, vdim, scale, chunk, base, rotated dims); right: (heads, dim, vdim, tau)."""
    h, kv, d, dv, scale, chunk, base, dims = left
    rh, rd, rdv, tau = right
    return {"type": "parallel", "mixer": {
        "left": {"heads": h, "kv_heads": kv, "dim": d, "vdim": dv, "scale": scale, "rot": {"base": base, "dims": dims}, "mask": {"size": chunk}},
        "right": {"heads": rh, "dim": rd, "vdim": rdv, "tau": tau}, "left_scale": left_scale, "right_scale": right_scale}}


def model(width, vocab, layers, loop=None, logit_scale=0.5, eps=1e-6):
    """``layers``: pairs of a mixer's entry and the feed-forward's size (None: none); ``loop``: (start, stop, times)."""
    out = {"architecture": "Salolorn", "vocab": vocab, "width": width, "norm": {"eps": eps}, "logit_scale": logit_scale,
           "layers": [dict(m, mlp=None if ff is None else {"kind": "dense", "ff": ff}) for m, ff in layers]}
    if loop is not None:
        out["loop"] = dict(zip(("start", "stop", "times"), loop))
    return out


CONFIGS = {
    # every mixer with and without a feed-forward; a loop in the middle whose passes hold every kind of cache and state
    "mixed": model(64, 97, [
        (delta(4, 2, 16, 24, 4), None), (latent(3, 16, 8, 12, 24, 0.3), 80),
        (parallel((4, 2, 16, 24, 0.3, 16, 500.0, 8), (2, 12, 20, 4.0), 0.7, 1.3), None), (delta(3, 3, 20, 16, 3), 40),
        (latent(2, 24, 4, 16, 16, 0.25, 100.0), None)], loop=(1, 4, 3), logit_scale=1.7),
    # sizes that are no multiples of 4, 8 or 16; one tap; a loop over every layer; one query/key head under five; a chunk of one
    "odd": model(48, 61, [
        (parallel((6, 1, 20, 12, 0.3, 7, 100.0, 6), (3, 10, 18, 16.0), -0.4, 0.9), 36), (delta(5, 1, 10, 13, 1), None),
        (parallel((3, 3, 8, 8, 0.6, 1, 50.0, 2), (1, 5, 7, 1.0), 1.0, 1.0), None), (delta(2, 2, 9, 6, 6), 24),
        (latent(5, 10, 6, 18, 20, 0.4, 1000.0), 40)], loop=(0, 5, 2), logit_scale=0.3, eps=1e-5),
    # no loop; heads of 64 and more in the recurrences, value heads wider and narrower than key heads, seventeen heads over
    # one latent (beyond a decode tile), a chunk longer than the prompts of most tests, layers of one kind in a row
    "wide": model(128, 128, [
        (delta(2, 1, 64, 128, 4), 128), (delta(2, 2, 96, 48, 2), None), (latent(17, 32, 32, 16, 32, 0.15), None),
        (parallel((4, 4, 64, 64, 0.12, 200, 250000.0, 32), (2, 64, 32, 8.0), 1.0, 0.5), 96)]),
    # a loop of one pass (its row of steps is added once) and one of the last layers
    "once": model(64, 80, [(latent(2, 16, 16, 16, 32, 0.25), 48), (delta(4, 2, 32, 32, 4), 64), (parallel((2, 1, 32, 16, 0.2, 24, 10000.0, 32), (2, 32, 40, 2.0), 1.5, -1.0), 48)],
                  loop=(1, 3, 1)),
}

# configurations for the GPU alone (the stand-ins would take minutes): sizes nearer a real model's layers
MORE_CONFIGS = {
    "big": model(512, 1000, [
        (delta(8, 4, 128, 128, 4), 512), (latent(8, 64, 32, 64, 128, 0.1), 768),
        (parallel((8, 2, 64, 128, 0.125, 96, 500000.0, 64), (4, 128, 64, 16.0), 0.8, 1.2), None), (delta(4, 2, 64, 256, 4), None),
        (parallel((4, 4, 128, 64, 0.088, 130, 10000.0, 32), (2, 64, 256, 8.0), 1.0, 1.0), 512)], loop=(2, 4, 2)),
}
CONFIGS_ALL = dict(CONFIGS, **MORE_CONFIGS)


def make_dir(tmp, name: str, seed: int = 0, sharpen: float = 3.0, dtype=torch.float32, rank: int = None) -> str:
    """A model folder of random weights, changed so that faults show: embeddings of order one, queries that make softmaxes far
    from flat (a key that is missing or one too many shows in the logits), sinks that take a good part of a softmax, step
    sizes, decays and gates that differ from token to token, rows of steps as large as the stream.  ``rank``: that of the
    linear attention's decays, in place of the random checkpoint's own."""
    from safetensors.torch import load_file, save_file
    from machserve_amd.weights import write_random_model
    out = os.path.join(str(tmp), f"salolorn_{name}_{seed}_{sharpen}_{rank}")
    write_random_model(dict(CONFIGS_ALL[name]), seed, out, dtype)
    path = os.path.join(out, "model.safetensors")
    w = load_file(path)
    g = torch.Generator().manual_seed(seed + 1)
    for k in sorted(w):
        t = w[k].float()
        of_order_one = 40.0 * (64.0 / t.shape[1]) ** 0.5 / 8.0 if t.dim() == 2 else 1.0
        if k == "embed":
            t = t * 40.0
        elif k == "loop.step":
            t = t * 60.0
        elif k.endswith(".left.q.norm") or k.endswith(".dkv.norm"):
            t = t * sharpen
        elif k.endswith(".sink"):
            t = t * 4.0 + 1.5
        elif k.endswith((".a1", ".a2")) and rank is not None:
            t = torch.randn((rank, t.shape[1]) if k.endswith("a1") else (t.shape[0], rank), generator=g) * (0.02 if k.endswith("a1") else 0.3)
            t = t * (of_order_one if k.endswith("a1") else 1.0)
        elif k.endswith(".a2.b"):
            t = t * 50.0 + 1.0
        elif k.endswith(".conv"):
            t = t * 2.0
        elif k.endswith(".dt_bias"):
            t = t + 1.0
        elif ".mix." in k and t.dim() == 2 and not k.endswith(".a2"):
            t = t * of_order_one
        elif k.endswith((".up", ".gate", ".down")):
            t = t * of_order_one
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
    """What a run keeps in its element type: operands of matrix products and the embedding."""
    return t.dim() == 2 and not name.endswith((".conv", ".a2", "loop.step"))


def within(got: torch.Tensor, want: torch.Tensor, dtype) -> bool:
    """float32: every row within rounding of sums taken in another order (a key too many or too few, a state that is lost or a
    pass without its row is off by 1e-2 and more).  bfloat16: rounding of activations grows through the layers, so half the
    rows must be within 4e-2; a row whose q or k comes out of its convolution next to nothing has that rounding multiplied
    by the unit norm: at most one row in sixty may be beyond 0.25 (logits that have nothing to do with the wanted ones are
    off by 1.4 in every row)."""
    e = relative_errors(got, want)
    if dtype == torch.float32:
        return float(e.max()) < 1e-4
    return float(e.median()) < 4e-2 and int((e > 0.25).sum()) <= max(1, e.numel() // 60)


def cut(rid, n, sizes):
    """One request of n tokens in portions of these sizes in turn."""
    out, at, k = [], 0, 0
    while at < n:
        c = min(sizes[k % len(sizes)], n - at)
        out.append([(rid, c)])
        at, k = at + c, k + 1
    return out
