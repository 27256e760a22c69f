"""A plain, slow Tevovik decoder for the tests to compare the engine with.

Whole sequences, no cache, no batching, one function per mechanism, in ordinary
tensor operations and explicit loops.  It shares no code with the package.
Computation is in `compute` (float64 by default) from the weights as stored.

The design: a token table times a constant plus a vector of sines and cosines of
the position; layers whose sublayers read the stream itself and whose results are
RMS-normed (weight stored around zero) on their way back into it; differential
attention (two softmax maps a head over the same values, the second taken off the
first lambda times, the difference normed per head) that sees the keys of its own
chunk of positions only and passes a gate per head, in some layers over the keys and values
of an earlier layer; a mixture of gated experts chosen among the best groups by
softmax scores; a final norm and an output matrix.
"""
from __future__ import annotations

import math
from typing import Callable, Dict, List, Optional, Sequence

import torch

# `rnd`: applied to every activation that one stage hands the next through memory in an implementation that keeps
# such hand-overs in 16 bits (never to the stream, a score, a softmax weight's sum, a norm's sum or the two maps'
# difference).  The identity by default.
_same = lambda x: x


def bf16_rounding(x: torch.Tensor) -> torch.Tensor:
    return x.to(torch.bfloat16).to(x.dtype)


def plain_unit(x: torch.Tensor, eps: float) -> torch.Tensor:
    """x over its root mean square."""
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)


def plain_norm(x: torch.Tensor, w: torch.Tensor, eps: float) -> torch.Tensor:
    """The norm of the stream's sublayers: its weight is stored as the distance from one."""
    return plain_unit(x, eps) * (1.0 + w)


def plain_positions(T: int, width: int, dtype=torch.float64) -> torch.Tensor:
    """[T, width]: feature 2i is the sine, feature 2i + 1 the cosine of position / 10000^(2i / width)."""
    out = torch.zeros(T, width, dtype=torch.float64)
    for c in range(width):
        rate = 10000.0 ** (-(c - c % 2) / width)
        for p in range(T):
            out[p, c] = math.cos(p * rate) if c % 2 else math.sin(p * rate)
    return out.to(dtype)


def plain_embed(table: torch.Tensor, tokens: Sequence[int], scale: float) -> torch.Tensor:
    x = table[torch.tensor(list(tokens), dtype=torch.long)] * scale
    return x + plain_positions(len(x), x.shape[1], x.dtype)


def plain_chunk_mask(T: int, size: int, dtype) -> torch.Tensor:
    """0 where position i sees position j, -inf elsewhere: j <= i, and both in the same stretch of `size` positions."""
    m = torch.full((T, T), float("-inf"), dtype=dtype)
    for i in range(T):
        m[i, i // size * size:i + 1] = 0.0
    return m


def plain_softmax(scores: torch.Tensor) -> torch.Tensor:
    e = torch.exp(scores - scores.max(dim=-1, keepdim=True).values)
    return e / e.sum(dim=-1, keepdim=True)


def plain_lambda(w: Dict[str, torch.Tensor], diff: float) -> torch.Tensor:
    return torch.exp((w["lq1"] * w["lk1"]).sum()) - torch.exp((w["lq2"] * w["lk2"]).sum()) + diff


def plain_difference(a1: torch.Tensor, a2: torch.Tensor, lam, diff: float, eps: float) -> torch.Tensor:
    """The two maps' outputs [.., vdim] of a head made one."""
    return plain_unit(a1 - lam * a2, eps) * (1.0 - diff)


def plain_keys_values(h: torch.Tensor, w: Dict[str, torch.Tensor], m: dict, eps: float):
    """(keys [T, kv_heads, 2, dim] after their norm, values [T, kv_heads, vdim])."""
    T, G, d, dv = h.shape[0], int(m["kv_heads"]), int(m["dim"]), int(m["vdim"])
    k = plain_unit((h @ w["k"].T).view(T, G, 2, d), eps) * w["k.norm"]
    return k, (h @ w["v"].T).view(T, G, dv)


def plain_attention(h: torch.Tensor, w: Dict[str, torch.Tensor], m: dict, eps: float, keys_values=None, rnd: Callable = _same):
    """Returns (output [T, width], (keys, values) as they were used).  keys_values: another layer's, or None for this
    layer's own."""
    T = h.shape[0]
    H, G, d, dv = int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"])
    q = rnd(plain_unit((h @ w["q"].T).view(T, H, 2, d), eps) * w["q.norm"])
    if keys_values is None:
        k, v = plain_keys_values(h, w, m, eps)
        keys_values = rnd(k), rnd(v)
    k, v = keys_values
    mask = plain_chunk_mask(T, int(m["mask"]["size"]), h.dtype)
    lam, diff = plain_lambda(w, float(m["diff"])), float(m["diff"])
    gate = 1.0 / (1.0 + torch.exp(-(h @ w["g"].T)))
    out = torch.zeros(T, H, dv, dtype=h.dtype)
    for head in range(H):
        g = head // (H // G)
        a = []
        for half in range(2):
            p = plain_softmax((q[:, head, half] @ k[:, g, half].T) * float(m["scale"]) + mask)
            a.append(rnd(p) @ v[:, g])
        out[:, head] = plain_difference(a[0], a[1], lam, diff, eps) * gate[:, head:head + 1]
    return rnd(out.reshape(T, H * dv)) @ w["o"].T, keys_values


def plain_route(z: torch.Tensor, top: int, groups: int, keep: int):
    """z: logits [T, experts].  (chosen experts, a list for each token; all experts' scores [T, experts])."""
    s = plain_softmax(z)
    T, E = s.shape
    per = E // groups
    chosen: List[List[int]] = []
    for t in range(T):
        row = s[t].tolist()
        best_of = [max(row[g * per:(g + 1) * per]) for g in range(groups)]
        kept = sorted(range(groups), key=lambda g: (-best_of[g], g))[:keep]
        open_to = [e for e in range(E) if e // per in kept]
        chosen.append(sorted(open_to, key=lambda e: (-row[e], e))[:top])
    return chosen, s


def plain_expert(h: torch.Tensor, w: Dict[str, torch.Tensor], weight, rnd: Callable = _same) -> torch.Tensor:
    """One expert's output times its weight (which multiplies the hidden activations: the down matrix is linear)."""
    g = h @ w["gate"].T
    return rnd(g / (1.0 + torch.exp(-g)) * (h @ w["up"].T) * weight) @ w["down"].T


def _under(tensors: Dict[str, torch.Tensor], prefix: str, compute=None) -> Dict[str, torch.Tensor]:
    return {n[len(prefix):]: (t if compute is None else t.to(compute)) for n, t in tensors.items() if n.startswith(prefix)}


def plain_experts(h: torch.Tensor, w: Dict[str, torch.Tensor], mlp: dict, rnd: Callable = _same) -> torch.Tensor:
    r = mlp["router"]
    groups = r.get("groups") or {"count": 1, "keep": 1}
    chosen, s = plain_route(h @ w["router"].T, int(r["top"]), int(groups["count"]), int(groups["keep"]))
    out = torch.zeros(h.shape[0], w["e0.down"].shape[0], dtype=h.dtype)
    for e in range(int(r["experts"])):
        rows = [t for t in range(h.shape[0]) if e in chosen[t]]
        if rows:
            out[rows] += plain_expert(h[rows], _under(w, f"e{e}."), s[rows, e:e + 1], rnd)
    return out


def plain_tevovik_logits(config: dict, tensors: Dict[str, torch.Tensor], tokens: Sequence[int], compute=torch.float64,
                         rnd: Callable = _same, after_layer: Optional[Callable] = None) -> torch.Tensor:
    """Logits [T, vocab] of the whole sequence.  `after_layer(i, x)` sees the stream after every layer."""
    eps = float(config["norm"]["eps"])
    x = plain_embed(tensors["embed"].to(compute), tokens, float(config["embedding"]["scale"]))
    kept = {}
    for i, layer in enumerate(config["layers"]):
        p, m = f"l{i}.", layer["mixer"]
        w = _under(tensors, p + "mix.", compute)
        y, kept[i] = plain_attention(rnd(x), w, m, eps, None if m.get("kv_from") is None else kept[int(m["kv_from"])], rnd)
        x = x + plain_norm(y, tensors[p + "norm1"].to(compute), eps)
        if layer.get("mlp") is not None:
            y = plain_experts(rnd(x), _under(tensors, p + "mlp.", compute), layer["mlp"], rnd)
            x = x + plain_norm(y, tensors[p + "norm2"].to(compute), eps)
        if after_layer is not None:
            after_layer(i, x)
    n = rnd(plain_norm(x, tensors["final.norm"].to(compute), eps))
    return n @ tensors["head"].to(compute).T
