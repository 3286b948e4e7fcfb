"""Plain, slow Salolorn decoder: whole sequences, no cache, one function per mechanism.

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
def rotate(x: torch.Tensor, base: float, dims: int, neighbours: bool) -> torch.Tensor:
    """``x [n, heads, d]``: of the first ``dims`` numbers of a head, pair i at position p turns by ``p base^(-2i / dims)``; the
    pairs are ``(2i, 2i + 1)`` (neighbours) or ``(i, i + dims / 2)``; the rest pass."""
    out = x.clone()
    for i in range(dims // 2):
        a, b = (2 * i, 2 * i + 1) if neighbours else (i, i + dims // 2)
        f = base ** (-2.0 * i / dims)
        for p in range(x.shape[0]):
            c, s = math.cos(p * f), math.sin(p * f)
            u, v = x[p, :, a], x[p, :, b]
            out[p, :, a] = u * c - v * s
            out[p, :, b] = v * c + u * s
    return out


# ------------------------------------------------------------------ attention
def causal_visible(n: int) -> torch.Tensor:
    return torch.arange(n)[None, :] <= torch.arange(n)[:, None]


def chunk_visible(n: int, size: int) -> torch.Tensor:
    """``[n, n]`` bool: row i sees j <= i of its own chunk of ``size`` positions, chunks counted from position 0."""
    i, j = torch.arange(n)[:, None], torch.arange(n)[None, :]
    return (j <= i) & ((i // size) == (j // size))


def sink_softmax(scores: torch.Tensor, see: torch.Tensor, sink=None) -> torch.Tensor:
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


def latent_attention(h: torch.Tensor, t: dict, p: str, m: dict, eps: float) -> torch.Tensor:
    """Every head's plain keys and values are maps of one normed latent per token; one rotated key part serves all heads."""
    n = h.shape[0]
    H, d, r, dv, rank = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    base = float(m["rot"]["base"])
    q = (h @ t[p + "q"].T).view(n, H, d + r)
    q_plain, q_rot = q[..., :d], rotate(q[..., d:], base, r, True)
    down = h @ t[p + "dkv"].T
    c = rms_norm(down[:, :rank], t[p + "dkv.norm"], eps)
    k_rot = rotate(down[:, None, rank:], base, r, True)[:, 0]
    k = (c @ t[p + "uk"].T).view(n, H, d)
    v = (c @ t[p + "uv"].T).view(n, H, dv)
    see = causal_visible(n)
    heads = []
    for a in range(H):
        w = sink_softmax((q_plain[:, a] @ k[:, a].T + q_rot[:, a] @ k_rot.T) * float(m["scale"]), see)
        heads.append(w @ v[:, a])
    return torch.cat(heads, 1) @ t[p + "o"].T


def chunked_attention(h: torch.Tensor, t: dict, p: str, m: dict, eps: float) -> torch.Tensor:
    """Grouped-query attention with a norm per head on q and k, chunks, a sink per head and a gate per head."""
    n = h.shape[0]
    H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = rms_norm((h @ t[p + "q"].T).view(n, H, d), t[p + "q.norm"], eps)
    k = rms_norm((h @ t[p + "k"].T).view(n, G, d), t[p + "k.norm"], eps)
    v = (h @ t[p + "v"].T).view(n, G, dv)
    base, dims = float(m["rot"]["base"]), int(m["rot"]["dims"])
    q, k = rotate(q, base, dims, False), rotate(k, base, dims, False)
    see = chunk_visible(n, int(m["mask"]["size"]))
    gate = torch.sigmoid(h @ t[p + "g"].T)
    heads = []
    for a in range(H):
        g = a // (H // G)
        w = sink_softmax(q[:, a] @ k[:, g].T * float(m["scale"]), see, t[p + "sink"][a])
        heads.append(w @ v[:, g] * gate[:, a:a + 1])
    return torch.cat(heads, 1) @ t[p + "o"].T


# ------------------------------------------------------------------ recurrences
def gated_linear_recurrence(q, k, v, alpha) -> torch.Tensor:
    """``S <- diag(alpha_t) S + k_t v_t^T``, ``o_t = S^T q_t`` per head from zero; q, k, alpha ``[n, H, d]``, v ``[n, H, dv]``."""
    n, H, d = q.shape
    S = torch.zeros(H, d, v.shape[-1], dtype=q.dtype)
    out = torch.empty_like(v)
    for i in range(n):
        S = alpha[i][:, :, None] * S + k[i][:, :, None] * v[i][:, None, :]
        out[i] = (S * q[i][:, :, None]).sum(1)
    return out


def gated_linear_attention(h: torch.Tensor, t: dict, p: str, m: dict, eps: float) -> torch.Tensor:
    n = h.shape[0]
    H, d, dv = m["heads"], m["dim"], m["vdim"]
    q = (h @ t[p + "q"].T).view(n, H, d) * d ** -0.5
    k = (h @ t[p + "k"].T).view(n, H, d)
    v = (h @ t[p + "v"].T).view(n, H, dv)
    z = (h @ t[p + "a1"].T) @ t[p + "a2"].T + t[p + "a2.b"]
    alpha = (torch.sigmoid(z) ** (1.0 / float(m["tau"]))).view(n, H, d)
    o = rms_norm(gated_linear_recurrence(q, k, v, alpha), t[p + "norm"], eps)
    return (o.reshape(n, H * dv) * silu(h @ t[p + "g"].T)) @ t[p + "o"].T


def causal_conv(x: torch.Tensor, w: torch.Tensor) -> torch.Tensor:
    """``y_t = sum_j w[:, j] x_(t - taps + 1 + j)`` per channel, zeros before the start."""
    n, taps = x.shape[0], w.shape[1]
    past = torch.cat([x.new_zeros(taps - 1, x.shape[1]), x], 0)
    return sum(past[j:j + n] * w[:, j] for j in range(taps))


def unit(x: torch.Tensor) -> torch.Tensor:
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


def delta_recurrence(q, k, v, beta, g) -> torch.Tensor:
    """``S <- g S; u = beta (v - S^T k); S <- S + k u^T; o = S^T q`` per head from zero; q, k ``[n, H, d]``, v ``[n, H, dv]``,
    beta, g ``[n, H]``."""
    n, H, d = q.shape
    S = torch.zeros(H, d, v.shape[-1], dtype=q.dtype)
    out = torch.empty_like(v)
    for i in range(n):
        S = g[i][:, None, None] * S
        u = beta[i][:, None] * (v[i] - (S * k[i][:, :, None]).sum(1))
        S = S + k[i][:, :, None] * u[:, None, :]
        out[i] = (S * q[i][:, :, None]).sum(1)
    return out


def gated_delta(h: torch.Tensor, t: dict, p: str, m: dict, eps: float) -> torch.Tensor:
    n = h.shape[0]
    H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k, v = (silu(causal_conv(h @ t[p + s].T, t[p + s + ".conv"])) for s in ("q", "k", "v"))
    of = torch.arange(H) // (H // G)
    q = (unit(q.view(n, G, d)) * d ** -0.5)[:, of]
    k = unit(k.view(n, G, d))[:, of]
    beta = torch.sigmoid(h @ t[p + "b"].T)
    g = torch.exp(-torch.exp(t[p + "A_log"]) * torch.nn.functional.softplus(h @ t[p + "a"].T + t[p + "dt_bias"], threshold=1e9))
    o = delta_recurrence(q, k, v.view(n, H, dv), beta, g)
    o = rms_norm(o, t[p + "norm"], eps).reshape(n, H * dv) * silu(h @ t[p + "g"].T)
    return o @ t[p + "o"].T


# ------------------------------------------------------------------ layers
def parallel(h: torch.Tensor, t: dict, p: str, m: dict, eps: float) -> torch.Tensor:
    """Two mixers that read the same input, weighted."""
    return (float(m["left_scale"]) * chunked_attention(h, t, p + "left.", m["left"], eps)
            + float(m["right_scale"]) * gated_linear_attention(h, t, p + "right.", m["right"], eps))


MIXERS = {"latent_attention": latent_attention, "parallel": parallel, "delta": gated_delta}


def feed_forward(h: torch.Tensor, t: dict, p: str) -> torch.Tensor:
    return (silu(h @ t[p + "gate"].T) * (h @ t[p + "up"].T)) @ t[p + "down"].T


def layer(x: torch.Tensor, t: dict, cfg: dict, i: int) -> torch.Tensor:
    """A norm before and one after each sublayer."""
    entry, eps, p = cfg["layers"][i], float(cfg["norm"]["eps"]), f"l{i}."
    y = MIXERS[entry["type"]](rms_norm(x, t[p + "norm1"], eps), t, p + "mix.", entry["mixer"], eps)
    x = x + rms_norm(y, t[p + "norm1b"], eps)
    if entry.get("mlp") is not None:
        x = x + rms_norm(feed_forward(rms_norm(x, t[p + "norm2"], eps), t, p + "mlp."), t[p + "norm2b"], eps)
    return x


def runs(cfg: dict) -> list:
    """The layer runs in order, each ``(layer, pass)`` with the pass it opens (None: it opens none)."""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return [(i, None) for i in range(n)]
    start, stop, times = int(loop["start"]), int(loop["stop"]), int(loop["times"])
    out = [(i, None) for i in range(start)]
    for k in range(times):
        out += [(i, k if i == start else None) for i in range(start, stop)]
    return out + [(i, None) for i in range(stop, n)]


def forward(tensors: dict, cfg: dict, tokens, dtype=torch.float64, layers_out: list = None) -> torch.Tensor:
    """Logits ``[n, vocab]`` of a whole sequence; ``layers_out`` receives the residual after every layer run."""
    t = {k: v.to(dtype) for k, v in tensors.items()}
    first = t["embed"][torch.as_tensor(tokens, dtype=torch.long)]
    x = first
    for i, opens in runs(cfg):
        if opens is not None:
            x = (x + first if opens > 0 else x) + t["loop.step"][opens]
        x = layer(x, t, cfg, i)
        if layers_out is not None:
            layers_out.append(x)
    return rms_norm(x, t["final.norm"], float(cfg["norm"]["eps"])) @ t["embed"].T * float(cfg["logit_scale"])


def greedy_generate(tensors: dict, cfg: dict, prompt, n_new: int, dtype=torch.float64) -> list:
    seq = list(prompt)
    for _ in range(n_new):
        seq.append(int(torch.argmax(forward(tensors, cfg, seq, dtype)[-1])))
    return seq[len(prompt):]
