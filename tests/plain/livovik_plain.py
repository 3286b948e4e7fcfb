"""Plain, slow Livovik decoder: whole sequences, no cache, one function per mechanism.

It shares no code with the engine.  Input is a dict of tensors by checkpoint name and the
config.json dict; everything is computed with ordinary torch operations on the CPU in
``dtype`` (float32 or float64).

Notation: ``n`` tokens, width ``w``; a linear map is ``y = x @ W.T`` with ``W [out, in]``.
"""
from __future__ import annotations

import math

import torch


def rms_norm(x: torch.Tensor, weight: torch.Tensor, eps: float) -> torch.Tensor:
    """Rows divided by ``sqrt(mean(x^2) + eps)``, times a weight per coordinate."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * weight


def silu(z: torch.Tensor) -> torch.Tensor:
    return z * torch.sigmoid(z)


# ------------------------------------------------------------------ rotation
def frequencies(rot: dict) -> list:
    """The pairs' frequencies ``base^(-2i / dims)``, slowed by wavelength if the rotation is scaled: those whose period is
    short beside the original context stay, those whose period is long are divided by the factor, and in between the two
    are mixed in proportion."""
    dims, base = int(rot["dims"]), float(rot["base"])
    out = []
    for i in range(dims // 2):
        f = base ** (-2.0 * i / dims)
        sc = rot.get("scaling")
        if sc:
            factor, low, high, original = (float(sc[k]) for k in ("factor", "low", "high", "original"))
            period = 2.0 * math.pi / f
            if period > original / low:
                f = f / factor
            elif period >= original / high:
                s = (original / period - low) / (high - low)
                f = (1.0 - s) * f / factor + s * f
        out.append(f)
    return out


def rotate(x: torch.Tensor, rot: dict) -> torch.Tensor:
    """``x [n, heads, d]``: of the first ``dims`` numbers of a head, the pair ``(i, i + dims / 2)`` at position p turns by
    ``p * f_i``; the rest pass."""
    half = int(rot["dims"]) // 2
    out = x.clone()
    for i, f in enumerate(frequencies(rot)):
        for p in range(x.shape[0]):
            c, s = math.cos(p * f), math.sin(p * f)
            u, v = x[p, :, i], x[p, :, i + half]
            out[p, :, i] = u * c - v * s
            out[p, :, i + half] = v * c + u * s
    return out


# ------------------------------------------------------------------ attention
def chunk_visible(n: int, size) -> torch.Tensor:
    """``[n, n]`` bool: row i sees j <= i of its own chunk of ``size`` positions (None: every j <= i), chunks counted from
    position 0."""
    i, j = torch.arange(n)[:, None], torch.arange(n)[None, :]
    see = j <= i
    return see & ((i // size) == (j // size)) if size else see


def sink_softmax(scores: torch.Tensor, see: torch.Tensor, sink) -> torch.Tensor:
    """Weights ``exp(s_j) / (exp(sink) + sum_j exp(s_j))`` over the seen keys; a sink of None is no term."""
    s = scores.masked_fill(~see, float("-inf"))
    m = s.max(-1, keepdim=True).values
    if sink is not None:
        m = torch.maximum(m, sink)
    e = torch.exp(s - m)
    total = e.sum(-1, keepdim=True)
    if sink is not None:
        total = total + torch.exp(sink - m)
    return e / total


def attention(h: torch.Tensor, t: dict, p: str, m: dict, eps: float) -> torch.Tensor:
    """Grouped-query attention with a norm per head on q and k, a rotation of part of a head, chunks, a sink per head and a
    gate per head.  ``t`` holds tensors whose names start with ``p``."""
    n = h.shape[0]
    H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = rms_norm((h @ t[p + "q"].T).view(n, H, d), t[p + "q.norm"], eps)
    k = rms_norm((h @ t[p + "k"].T).view(n, G, d), t[p + "k.norm"], eps)
    v = (h @ t[p + "v"].T).view(n, G, dv)
    if m.get("rot"):
        q, k = rotate(q, m["rot"]), rotate(k, m["rot"])
    see = chunk_visible(n, int(m["mask"]["size"]) if m.get("mask") else None)
    gate = torch.sigmoid(h @ t[p + "g"].T)
    heads = []
    for a in range(H):
        g = a // (H // G)
        w = sink_softmax(q[:, a] @ k[:, g].T * float(m["scale"]), see, t[p + "sink"][a])
        heads.append(w @ v[:, g] * gate[:, a:a + 1])
    return torch.cat(heads, 1) @ t[p + "o"].T


# ------------------------------------------------------------------ feed-forwards
def dense(h: torch.Tensor, t: dict, p: str) -> torch.Tensor:
    """Two layers around the square of relu."""
    return torch.relu(h @ t[p + "up"].T) ** 2 @ t[p + "down"].T


def expert(x: torch.Tensor, t: dict, p: str) -> torch.Tensor:
    return (silu(x @ t[p + "gate"].T) * (x @ t[p + "up"].T)) @ t[p + "down"].T


def route(h: torch.Tensor, t: dict, p: str, top: int):
    """The chosen experts ``[n, top]`` and their weights: the largest sigmoid scores, not divided by their sum."""
    s = torch.sigmoid(h @ t[p + "router"].T)
    w, idx = torch.topk(s, top, dim=-1)
    return idx, w


def moe(h: torch.Tensor, t: dict, p: str, mlp: dict) -> torch.Tensor:
    """Each chosen expert runs on its weight times the row; an expert for every token is gated by one number a row."""
    idx, w = route(h, t, p, int(mlp["router"]["top"]))
    rows = []
    for i in range(h.shape[0]):
        y = torch.zeros_like(h[i:i + 1])
        for e, g in zip(idx[i].tolist(), w[i]):
            y = y + expert(g * h[i:i + 1], t, f"{p}e{e}.")
        rows.append(y)
    out = torch.cat(rows, 0)
    if mlp.get("shared"):
        out = out + expert(h, t, p + "shared.") * torch.sigmoid(h @ t[p + "shared.sg"].T)
    return out


def feed_forward(h: torch.Tensor, t: dict, p: str, mlp: dict) -> torch.Tensor:
    return dense(h, t, p) if mlp["kind"] == "dense" else moe(h, t, p, mlp)


# ------------------------------------------------------------------ the model
def owner(layers: list, i: int) -> int:
    """The layer whose tensors layer i uses."""
    while layers[i].get("weights_of") is not None:
        i = layers[i]["weights_of"]
    return i


def layer(x: torch.Tensor, t: dict, cfg: dict, i: int) -> torch.Tensor:
    """One layer: norms after the sums, the sublayers reading x itself."""
    entry, eps, alpha = cfg["layers"][i], float(cfg["norm"]["eps"]), float(cfg["postln_alpha"])
    p = f"l{owner(cfg['layers'], i)}."
    x = rms_norm(alpha * x + attention(x, t, p + "mix.", entry["mixer"], eps), t[p + "norm1"], eps)
    if entry.get("mlp") is not None:
        x = rms_norm(alpha * x + feed_forward(x, t, p + "mlp.", entry["mlp"]), t[p + "norm2"], eps)
    return x


def forward(tensors: dict, cfg: dict, tokens, dtype=torch.float64, layers_out: list = None) -> torch.Tensor:
    """Logits ``[n, vocab]`` of a whole sequence; ``layers_out`` receives the residual after every layer."""
    t = {k: v.to(dtype) for k, v in tensors.items()}
    x = t["embed"][torch.as_tensor(tokens, dtype=torch.long)]
    for i in range(len(cfg["layers"])):
        x = layer(x, t, cfg, i)
        if layers_out is not None:
            layers_out.append(x)
    return rms_norm(x, t["final.norm"], float(cfg["norm"]["eps"])) @ t["head"].T


def greedy_generate(tensors: dict, cfg: dict, prompt, n_new: int, dtype=torch.float64) -> list:
    seq = list(prompt)
    for _ in range(n_new):
        seq.append(int(torch.argmax(forward(tensors, cfg, seq, dtype)[-1])))
    return seq[len(prompt):]
