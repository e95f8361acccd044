"""A plain, slow Mesolix: whole sequences at once, no cache, one function per mechanism, in the precision of the
tensors it is given (tests hand it 64-bit ones).  It shares no code with the engine.

Notation: ``h`` [T, D] rows of one sequence, positions 0..T-1; tensors under their checkpoint names in a dict ``w``;
a layer's description as config.json gives it."""

from __future__ import annotations

from typing import Dict, List, Optional

import torch


# ----------------------------------------------------------------------------- small pieces
def over_rms(x, eps: float):
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)


def rms_norm(x, weight, eps: float):
    return over_rms(x, eps) * weight


def shifted_norm(x, weight, eps: float):
    """The norms before the branches and before the head: their weight is stored around zero."""
    return over_rms(x, eps) * (1.0 + weight)


def silu(z):
    return z * torch.sigmoid(z)


def causal(T: int):
    """bool [T, T]: query i sees key j <= i."""
    i = torch.arange(T)
    return i[None, :] <= i[:, None]


def within(T: int, size: int):
    """bool [T, T]: query i sees key j when 0 <= i - j < size."""
    dist = torch.arange(T)[:, None] - torch.arange(T)[None, :]
    return (dist >= 0) & (dist < size)


# ----------------------------------------------------------------------------- attention through a latent
def softmax_with_sink(s, sink):
    """``exp(s_j) / (exp(sink) + sum_j exp(s_j))`` over the last axis of ``s`` [H, T, T], a sink a head."""
    top = torch.maximum(s.max(dim=-1, keepdim=True).values, sink[:, None, None])
    e = torch.exp(s - top)
    return e / (e.sum(dim=-1, keepdim=True) + torch.exp(sink[:, None, None] - top))


def latent_attention(h, w, p: str, m: Dict, eps: float):
    """Keys and values of all heads expanded from one normed latent per token, queries from a normed latent of their
    own, a sink in the denominator, the heads gated channel by channel."""
    T, H, d, dv = h.shape[0], m["heads"], m["dim"], m["vdim"]
    cq = rms_norm(h @ w[p + "dq"].T, w[p + "dq.norm"], eps)
    c = rms_norm(h @ w[p + "dkv"].T, w[p + "dkv.norm"], eps)
    q = (cq @ w[p + "uq"].T).view(T, H, d)
    k = (c @ w[p + "uk"].T).view(T, H, d)
    v = (c @ w[p + "uv"].T).view(T, H, dv)
    s = (torch.einsum("ihd,jhd->hij", q, k) * m["scale"]).masked_fill(~causal(T)[None], float("-inf"))
    o = torch.einsum("hij,jhd->ihd", softmax_with_sink(s, w[p + "sink"]), v).reshape(T, H * dv)
    return (o * torch.sigmoid(h @ w[p + "g"].T)) @ w[p + "o"].T


# ----------------------------------------------------------------------------- windowed attention with bucketed distances
def bucket(n: int, rows: int, most: int) -> int:
    """The row of the table for a distance n: one row a distance below rows/2, then logarithmic up to ``most``.  The
    floor of ``ln(n / half) / ln(most / half) * (rows - half)`` is taken in whole numbers: the largest t with
    ``(most / half)^t <= (n / half)^(rows - half)``."""
    half = rows // 2
    if n < half:
        return n
    steps, t = rows - half, 0
    while half + t + 1 < rows and most ** (t + 1) * half ** steps <= n ** steps * half ** (t + 1):
        t += 1
    return min(rows - 1, half + t)


def distance_bias(rel, T: int, most: int):
    """``[H, T, T]`` with ``rel[bucket(i - j), h]`` for j <= i (0 elsewhere)."""
    rows = [bucket(n, rel.shape[0], most) for n in range(T)]
    by_distance = rel[torch.tensor(rows)]  # [T, H]
    dist = (torch.arange(T)[:, None] - torch.arange(T)[None, :])
    return torch.where((dist >= 0)[None], by_distance[dist.clamp(min=0)].permute(2, 0, 1), torch.zeros((), dtype=rel.dtype))


def windowed_attention(h, w, p: str, m: Dict):
    """Grouped-query attention inside a sliding window, a learned bias by distance, the heads gated channel by channel."""
    T, H, G, d, dv = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = (h @ w[p + "q"].T).view(T, H, d)
    k = (h @ w[p + "k"].T).view(T, G, d).repeat_interleave(H // G, dim=1)
    v = (h @ w[p + "v"].T).view(T, G, dv).repeat_interleave(H // G, dim=1)
    s = torch.einsum("ihd,jhd->hij", q, k) * m["scale"] + distance_bias(w[p + "rel"], T, m["bias_max"])
    s = s.masked_fill(~within(T, m["mask"]["size"])[None], float("-inf"))
    o = torch.einsum("hij,jhd->ihd", torch.softmax(s, dim=-1), v).reshape(T, H * dv)
    return (o * torch.sigmoid(h @ w[p + "g"].T)) @ w[p + "o"].T


# ----------------------------------------------------------------------------- the state-space mixer
def causal_conv(x, taps, bias):
    """``out[t, c] = bias[c] + sum_j taps[c, j] x[t - (K - 1 - j), c]``, zeros before the start."""
    K = taps.shape[1]
    padded = torch.cat([x.new_zeros(K - 1, x.shape[1]), x])
    return bias + sum(padded[j : j + x.shape[0]] * taps[:, j] for j in range(K))


def ssd_states(x, B, C, dt, log_a):
    """Per head ``S_t = exp(dt a) S_(t-1) + dt B_t x_t^T; y_t = S_t^T C_t`` from a zero state; x [T, H, dv], B and C
    [T, H, N], dt [T, H], ``a = -exp(log_a)`` [H] -> y [T, H, dv]."""
    S = x.new_zeros(x.shape[1], B.shape[2], x.shape[2])
    out = []
    for t in range(x.shape[0]):
        keep = torch.exp(-torch.exp(log_a) * dt[t])
        S = keep[:, None, None] * S + dt[t][:, None, None] * B[t][:, :, None] * x[t][:, None, :]
        out.append(torch.einsum("hnv,hn->hv", S, C[t]))
    return torch.stack(out)


def softplus(z):
    return torch.where(z > 0, z, torch.zeros_like(z)) + torch.log1p(torch.exp(-z.abs()))


def state_space(h, w, p: str, m: Dict, eps: float):
    """A state-space layer whose heads have one decay each, over short convolutions of x, B and C; gated, then normed in
    equal parts."""
    T, H, dv, N, G = h.shape[0], m["heads"], m["vdim"], m["state"], m["groups"]
    inner = H * dv
    z, xbc, dt = (h @ w[p + "in"].T).split([inner, inner + 2 * G * N, H], dim=1)
    xbc = silu(causal_conv(xbc, w[p + "conv"], w[p + "conv.b"]))
    x, B, C = xbc.split([inner, G * N, G * N], dim=1)
    x = x.view(T, H, dv)
    B, C = (u.view(T, G, N).repeat_interleave(H // G, dim=1) for u in (B, C))
    dt = softplus(dt + w[p + "dt_bias"])
    y = ssd_states(x, B, C, dt, w[p + "A_log"]) + w[p + "D"][None, :, None] * x
    y = y.reshape(T, inner) * silu(z)
    y = over_rms(y.view(T, m["norm_groups"], -1), eps).reshape(T, inner) * w[p + "norm"]
    return y @ w[p + "o"].T


# ----------------------------------------------------------------------------- feed-forward
def clamped_glu(h, w, p: str, limit: float):
    g = torch.clamp(h @ w[p + "gate"].T, max=limit)
    u = torch.clamp(h @ w[p + "up"].T, -limit, limit)
    return (g * torch.sigmoid(1.702 * g) * (u + 1.0)) @ w[p + "down"].T


def expert(h, w, p: str):
    return (silu(h @ w[p + "gate"].T) * (h @ w[p + "up"].T)) @ w[p + "down"].T


def routed_choice(z, top: int):
    """``(chosen experts [T, top], weights)``: the largest scores ``sigmoid(z)``, which are the weights as they are."""
    best = torch.sigmoid(z).topk(top, dim=-1)
    return best.indices, best.values


def mixture(h, w, p: str, mlp: Dict):
    """A chosen expert works on the input times its weight; its output is added as it is."""
    ids, weights = routed_choice(h @ w[p + "router"].T, mlp["router"]["top"])
    out = expert(h, w, p + "shared.") if mlp.get("shared") else torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, g in zip(ids[t].tolist(), weights[t]):
            out[t] += expert(g * h[t : t + 1], w, f"{p}e{e}.")[0]
    return out


def feed_forward(h, w, i: int, mlp: Dict):
    if mlp["kind"] == "dense":
        return clamped_glu(h, w, f"l{i}.mlp.", mlp["limit"])
    return mixture(h, w, f"l{i}.mlp.", mlp)


# ----------------------------------------------------------------------------- the model
def owner(config: Dict, i: int) -> int:
    """The layer whose tensors layer i uses."""
    while config["layers"][i].get("weights_of") is not None:
        i = config["layers"][i]["weights_of"]
    return i


def mix(h, w, i: int, entry: Dict, eps: float):
    p, m = f"l{i}.mix.", entry["mixer"]
    if entry["type"] == "latent_attention":
        return latent_attention(h, w, p, m, eps)
    if entry["type"] == "mamba2":
        return state_space(h, w, p, m, eps)
    return windowed_attention(h, w, p, m)


def layer(x, w, i: int, entry: Dict, eps: float):
    x = x + mix(shifted_norm(x, w[f"l{i}.norm1"], eps), w, i, entry, eps)
    if entry.get("mlp") is not None:
        x = x + feed_forward(shifted_norm(x, w[f"l{i}.norm2"], eps), w, i, entry["mlp"])
    return x


def forward(config: Dict, tensors: Dict[str, torch.Tensor], tokens: List[int], dtype=torch.float64, layer_outputs: Optional[list] = None):
    """Logits [T, vocab] of one sequence; ``layer_outputs`` receives the stream after every layer."""
    w = {k: (v.to(dtype) if v.is_floating_point() else v) for k, v in tensors.items()}
    eps = float(config["norm"]["eps"])
    x = w["embed"][torch.tensor(tokens, dtype=torch.long)] + w["pos"][: len(tokens)]
    for i, entry in enumerate(config["layers"]):
        x = layer(x, w, owner(config, i), entry, eps)
        if layer_outputs is not None:
            layer_outputs.append(x)
    return shifted_norm(x, w["final.norm"], eps) @ w["head"].T
