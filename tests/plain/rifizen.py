"""A plain, slow Rifizen: whole sequences at once, no cache, one function per mechanism, in the precision of the
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


def silu(z):
    return z * torch.sigmoid(z)


def rotate_half(x, positions, dims: int, base: float):
    """The first ``dims`` channels of the last axis of ``x`` [T, H, d] turned by their position's angles, channel i
    with channel i + dims/2; the others pass."""
    if dims == 0:
        return x
    i = torch.arange(dims // 2, dtype=torch.float64)
    ang = positions.to(torch.float64)[:, None] * (float(base) ** (-2.0 * i / dims))[None, :]
    c, s = torch.cos(ang).to(x.dtype)[:, None, :], torch.sin(ang).to(x.dtype)[:, None, :]
    out = x.clone()
    u, v = x[..., : dims // 2], x[..., dims // 2 : dims]
    out[..., : dims // 2] = u * c - v * s
    out[..., dims // 2 : dims] = v * c + u * s
    return out


def slopes(heads: int, dtype=torch.float64):
    """What a token of distance costs head h: ``2^(-8 (h + 1) / heads)``."""
    return torch.tensor([2.0 ** (-8.0 * (h + 1) / heads) for h in range(heads)], dtype=torch.float64).to(dtype)


def visible(T: int, size: int):
    """bool [T, T]: query i sees key j when 0 <= i - j < size."""
    dist = torch.arange(T)[:, None] - torch.arange(T)[None, :]
    return (dist >= 0) & (dist < size)


def biased_scores(q, k, scale: float, cap: float):
    """q, k [T, H, d] -> [H, T, T]: capped scores less the slope times the distance."""
    T, H = q.shape[0], q.shape[1]
    s = torch.einsum("ihd,jhd->hij", q, k) * scale
    s = cap * torch.tanh(s / cap)
    dist = (torch.arange(T)[:, None] - torch.arange(T)[None, :]).to(q.dtype)
    return s - slopes(H, q.dtype)[:, None, None] * dist[None]


# ----------------------------------------------------------------------------- the two mixers
def biased_attention(h, w, p: str, m: Dict, eps: float):
    """Grouped-query attention inside a sliding window: unit-RMS queries and keys, no rotation, a cap, a bias by
    distance."""
    T = h.shape[0]
    H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = over_rms((h @ w[p + "q"].T).view(T, H, d), eps)
    k = over_rms((h @ w[p + "k"].T).view(T, G, d), eps).repeat_interleave(H // G, dim=1)
    v = (h @ w[p + "v"].T).view(T, G, dv).repeat_interleave(H // G, dim=1)
    s = biased_scores(q, k, m["scale"], m["softcap"]).masked_fill(~visible(T, m["mask"]["size"])[None], float("-inf"))
    o = torch.einsum("hij,jhd->ihd", torch.softmax(s, dim=-1), v)
    return o.reshape(T, H * dv) @ w[p + "o"].T


def retention_states(q, k, v, decay):
    """Per head ``S <- decay S + k v^T; o = S^T q`` from a zero state; q, k [T, H, d], v [T, H, dv] -> o [T, H, dv]."""
    S = q.new_zeros(q.shape[1], q.shape[2], v.shape[2])
    keep = torch.as_tensor(decay, dtype=torch.float64).to(q.dtype)[:, None, None]
    out = []
    for t in range(q.shape[0]):
        S = keep * S + k[t][:, :, None] * v[t][:, None, :]
        out.append(torch.einsum("hdv,hd->hv", S, q[t]))
    return torch.stack(out)


def retention(h, w, p: str, m: Dict, eps: float):
    """Linear attention whose state fades by a constant per head; rotated q and k, k times d^-1/2; every head over its
    root mean square, times the gate."""
    T = h.shape[0]
    H, d, dv = m["heads"], m["dim"], m["vdim"]
    pos = torch.arange(T)
    q = rotate_half((h @ w[p + "q"].T).view(T, H, d), pos, m["rot"]["dims"], m["rot"]["base"])
    k = rotate_half((h @ w[p + "k"].T).view(T, H, d), pos, m["rot"]["dims"], m["rot"]["base"]) * d ** -0.5
    v = (h @ w[p + "v"].T).view(T, H, dv)
    o = over_rms(retention_states(q, k, v, m["decay"]), eps)
    return (o.reshape(T, H * dv) * silu(h @ w[p + "g"].T)) @ w[p + "o"].T


def pair(h, w, i: int, m: Dict, eps: float):
    """Half the sum of the two mixers' results, each normed over the width with a weight of its own."""
    left = rms_norm(biased_attention(h, w, f"l{i}.mix.left.", m["left"], eps), w[f"l{i}.mix.left.out"], eps)
    right = rms_norm(retention(h, w, f"l{i}.mix.right.", m["right"], eps), w[f"l{i}.mix.right.out"], eps)
    return 0.5 * (left + right)


# ----------------------------------------------------------------------------- feed-forward
def dense(h, w, p: str):
    return torch.relu(h @ w[p + "up"].T) ** 2 @ w[p + "down"].T


def expert(h, w, p: str):
    return (silu(h @ w[p + "gate"].T) * (h @ w[p + "up"].T)) @ w[p + "down"].T


def routed_choice(z, top: int):
    """``(chosen experts [T, top], weights)``: the largest of z, and the softmax over those alone."""
    best = z.topk(top, dim=-1)
    return best.indices, torch.softmax(best.values, dim=-1)


def mixture(h, w, p: str, mlp: Dict):
    ids, weights = routed_choice(h @ w[p + "router"].T + w[p + "router.b"], mlp["router"]["top"])
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, g in zip(ids[t].tolist(), weights[t]):
            out[t] += g * expert(h[t : t + 1], w, f"{p}e{e}.")[0]
    return out


def feed_forward(h, w, i: int, mlp: Dict):
    return dense(h, w, f"l{i}.mlp.") if mlp["kind"] == "dense" else mixture(h, w, f"l{i}.mlp.", mlp)


# ----------------------------------------------------------------------------- the model
def run_order(config: Dict) -> List[tuple]:
    """``(layer, pass whose vector is added before it or None)`` in the order of execution."""
    n, loop = len(config["layers"]), config.get("loop")
    if not loop:
        return [(i, None) for i in range(n)]
    order = [(i, None) for i in range(loop["start"])]
    for t in range(loop["times"]):
        order += [(i, t if i == loop["start"] else None) for i in range(loop["start"], loop["stop"])]
    return order + [(i, None) for i in range(loop["stop"], n)]


def layer(x, w, i: int, entry: Dict, eps: float):
    x = x + rms_norm(pair(rms_norm(x, w[f"l{i}.norm1"], eps), w, i, entry["mixer"], eps), w[f"l{i}.norm1b"], eps)
    if entry.get("mlp") is not None:
        x = x + rms_norm(feed_forward(rms_norm(x, w[f"l{i}.norm2"], eps), w, i, entry["mlp"]), w[f"l{i}.norm2b"], eps)
    return x


def forward(config: Dict, tensors: Dict[str, torch.Tensor], tokens: List[int], dtype=torch.float64, layer_outputs: Optional[list] = None):
    """Logits [T, vocab] of one sequence; ``layer_outputs`` receives the stream after every layer run."""
    w = {k: (v.to(dtype) if v.is_floating_point() else v) for k, v in tensors.items()}
    eps = float(config["norm"]["eps"])
    x = w["embed"][torch.tensor(tokens, dtype=torch.long)]
    for i, step in run_order(config):
        if step is not None:
            x = x + w["loop.step"][step]
        x = layer(x, w, i, config["layers"][i], eps)
        if layer_outputs is not None:
            layer_outputs.append(x)
    return rms_norm(x, w["final.norm"], eps) @ w["head"].T
