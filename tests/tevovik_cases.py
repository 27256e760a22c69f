"""Small Tevovik configurations for the tests, their random weights, and the comparison with the plain decoder.

The configurations differ from one another in every size and option: one, several or all query heads to a key head, maps
narrower and wider than the values, chunks shorter and longer than a page and of sizes that are multiples of nothing,
layers that read an earlier layer's keys through a chunk shorter or longer than that layer's own, routers with and without
groups, layers without a feed-forward, widths that are odd.
"""
from __future__ import annotations

import os
from typing import Dict, List

import torch

from llm_rs_amd import TevovikConfig, random_model_tensors, write_model_folder
from plain_tevovik import bf16_rounding, plain_tevovik_logits


def moe(experts, top, ff, groups=None):
    return {"kind": "moe", "expert": {"ff": ff},
            "router": {"experts": experts, "top": top, "groups": None if groups is None else {"count": groups[0], "keep": groups[1]}}}


def attention(heads, kv_heads, dim, vdim, chunk, scale=None, diff=0.4, kv_from=None, mlp=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": 2.0 * dim ** -0.5 if scale is None else scale,
         "diff": diff, "mask": {"size": chunk}}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "attention", "mixer": m, "mlp": mlp}


def config(width, vocab, layers, eps=1e-5, scale=1.7):
    return {"architecture": "Tevovik", "vocab": vocab, "width": width, "embedding": {"scale": scale}, "norm": {"eps": eps}, "layers": layers}


ODD = config(45, 97, [
    attention(6, 2, 5, 6, 13, mlp=moe(6, 2, 7, (3, 2))),
    attention(3, 3, 9, 20, 50, diff=0.15),
    attention(2, 2, 5, 6, 13, kv_from=0, mlp=moe(5, 1, 9)),
    attention(4, 2, 5, 6, 29, kv_from=0, diff=0.8, mlp=moe(4, 4, 6, (2, 2))),
    attention(1, 1, 11, 3, 7, mlp=moe(8, 3, 5, (4, 3))),
    attention(9, 3, 9, 20, 10, kv_from=1, mlp=moe(3, 2, 4)),
])
PLAIN = config(64, 128, [
    attention(4, 2, 16, 32, 32, mlp=moe(8, 2, 24, (2, 1))),
    attention(8, 2, 16, 32, 32, kv_from=0, diff=0.6, mlp=moe(6, 3, 16)),
    attention(2, 2, 16, 16, 40, mlp=moe(4, 1, 32, (4, 2))),
    attention(2, 1, 32, 48, 24),
], eps=1e-6)
# widths at which the bfloat16 products go to the matrix cores, heads and values the matrix-core attention takes
WIDE = config(384, 352, [
    attention(8, 2, 32, 64, 80, mlp=moe(8, 2, 96, (4, 2))),
    attention(6, 2, 64, 128, 48, diff=0.2, mlp=moe(4, 2, 128)),
    attention(16, 2, 32, 64, 130, kv_from=0, mlp=moe(12, 3, 64, (3, 1))),
    attention(4, 4, 64, 64, 33),
    attention(8, 1, 128, 256, 64, mlp=moe(6, 1, 64, (2, 2))),
    attention(2, 2, 64, 128, 100, kv_from=1, diff=0.7, mlp=moe(5, 5, 32)),
])
CONFIGS = {"odd": ODD, "plain": PLAIN, "wide": WIDE}
PAGE_SIZE = {"odd": 4, "plain": 16, "wide": 16}


def one_layer(layer, width=40, vocab=61, eps=1e-5):
    return config(width, vocab, [layer], eps)


def loud(tensors) -> None:
    """Random weights under which what a token is shows: its row of the table as large as the position vector, lambdas
    that differ from layer to layer, and routers enlarged so that the choice of experts is no near tie."""
    for name in list(tensors):
        factor = (50.0 if name == "embed" else 4.0 if name.endswith((".lq1", ".lk1", ".lq2", ".lk2")) else 40.0 if name.endswith(".mlp.router")
                  else 10.0 if name.endswith(".mix.g") else None)
        if factor is not None:
            tensors[name] = (tensors[name].double() * factor).to(tensors[name].dtype)


def calm_routers(tensors) -> None:
    """Routers under which 16-bit rounding of their input cannot change which experts a token gets (two scores that differ
    by less than the rounding would otherwise fall either way, and an expert swapped for another is no rounding error):
    one feature of the stream is made nearly the same for every token (the same in every row of the table, of a slow wave
    of the position, and left alone by every norm on the way into the stream), and the routers read their experts' order
    from it and hardly anything from the rest.  Which experts a token gets by its own scores is what the 32-bit runs
    check."""
    width = tensors["embed"].shape[1]
    at = width - 1 if width % 2 == 0 else width - 2          # (the slowest cosine)
    tensors["embed"][:, at] = 1.0
    for name in list(tensors):
        if name.endswith((".norm1", ".norm2")):
            tensors[name][at] = -1.0
        elif name.endswith(".mlp.router"):
            n = tensors[name].shape[0]
            tensors[name] = (tensors[name].double() * 0.002).to(tensors[name].dtype)
            order = torch.tensor([(5 * e + 2) % n if n % 5 else (3 * e + 1) % n for e in range(n)], dtype=torch.float64)
            if len(set(order.tolist())) < n:
                order = torch.arange(n, dtype=torch.float64)
            tensors[name][:, at] = (0.12 * order).to(tensors[name].dtype)


def make_model(cfg: dict, seed: int = 0, change=None, calm_router: bool = False):
    """(typed config, {name: bfloat16 tensor}); `change(tensors)` may put values of its own in."""
    typed = TevovikConfig.from_dict(cfg)
    tensors = random_model_tensors(typed, seed)
    loud(tensors)
    if calm_router:
        calm_routers(tensors)
    if change is not None:
        change(tensors)
    return typed, tensors


def make_folder(tmp_path, cfg: dict, seed: int = 0, change=None, name: str = "model", calm_router: bool = False) -> str:
    typed, tensors = make_model(cfg, seed, change, calm_router)
    folder = os.path.join(str(tmp_path), name)
    write_model_folder(folder, typed, tensors)
    return folder


def reference(cfg: dict, tensors, requests: Dict[str, List[int]], rnd=None):
    kw = {} if rnd is None else {"rnd": rnd}
    return {rid: plain_tevovik_logits(cfg, tensors, toks, **kw) for rid, toks in requests.items()}


def allowed_error(dtype: str, cfg: dict, tensors, requests, exact) -> float:
    """How far the engine may be from the exact logits, as a part of a sequence's largest logit.  float32: 3e-5, or four times
    as far as the plain decoder itself gets in 32-bit where that is more: where the two maps of a head nearly cancel, the
    norm of their difference enlarges what rounding left of it, by much at a few positions (the plain decoder's own figure
    at such a position moves by a factor of two and a half from one machine's order of sums to another's).  bfloat16: twice as far as the plain decoder gets when every
    activation that passes through memory between two stages is rounded to bfloat16 (the engine keeps some of those in
    32-bit and sums in other orders; it does not round more often)."""
    kw = {"compute": torch.float32} if dtype == "float32" else {"rnd": bf16_rounding}
    other = {rid: plain_tevovik_logits(cfg, tensors, toks, **kw).double() for rid, toks in requests.items()}
    far = max(float((other[r] - exact[r]).abs().max()) / float(exact[r].abs().max()) for r in requests)
    return max(3e-5, 4.0 * far) if dtype == "float32" else 2.0 * far


def check_rows(rows, exact, requests, allowed: float, what: str = "") -> float:
    """Every position of every request within `allowed` of the exact logits."""
    worst = 0.0
    for rid, toks in requests.items():
        ref = exact[rid]
        scale = float(ref.abs().max())
        assert sorted(rows[rid]) == list(range(len(toks))), f"{what} request {rid}: not every position came back"
        got = torch.stack([rows[rid][p] for p in range(len(toks))]).double()
        assert torch.isfinite(got).all(), f"{what} request {rid}: logits that are not numbers"
        err = (got - ref).abs().max(dim=1).values / scale
        bad = (err > allowed).nonzero()
        assert len(bad) == 0, (f"{what} request {rid}: first wrong position {int(bad[0])} of {len(toks)} (error "
                               f"{float(err[int(bad[0])]):.3e} of the largest logit, allowed {allowed:.1e}); {len(bad)} positions wrong")
        worst = max(worst, float(err.max()))
    return worst


MARK = 7


def marked_model(heads, kv_heads, dim, vdim, chunk, second_chunk=None, width=48, vocab=50, loudness=14.0):
    """One layer in which the first map's key of token MARK stands out for every query, wherever it stands, while the
    second map sees all keys of the chunk alike.  Two features of the stream are the same for every token but for that one
    (the waves of the position on them are slow): the last one is 4 times the table's scale for all, and every query reads
    it alone; the one before it is large in the marked token's row only, and the last feature of the first map's keys reads
    it alone.  second_chunk: a second layer follows that reads the first's keys through a chunk of that size."""
    layers = [attention(heads, kv_heads, dim, vdim, chunk, scale=loudness / dim)]
    if second_chunk is not None:
        layers.append(attention(heads, kv_heads, dim, vdim, second_chunk, scale=loudness / dim, kv_from=0))
    cfg = config(width, vocab, layers)

    def change(t):
        t["embed"][:, width - 2], t["embed"][:, width - 1] = 0.0, 4.0
        t["embed"][MARK, width - 2] = 30.0
        wk = t["l0.mix.k"].double().view(kv_heads, 2, dim, width)
        wk[:, :, :, width - 2] = 0.0
        wk[:, :, dim - 1, :] = 0.0
        wk[:, 0, dim - 1, width - 2] = 1.0
        t["l0.mix.k"] = wk.reshape(-1, width).to(torch.bfloat16)
        t["l0.mix.k.norm"] = torch.ones_like(t["l0.mix.k.norm"])
        for i in range(len(layers)):
            t[f"l{i}.norm1"][width - 2:] = -1.0          # (no sublayer touches the two features)
            wq = torch.zeros(heads, 2, dim, width, dtype=torch.float64)
            wq[:, :, dim - 1, width - 1] = 1.0
            t[f"l{i}.mix.q"] = wq.reshape(-1, width).to(torch.bfloat16)
            t[f"l{i}.mix.q.norm"] = torch.ones_like(t[f"l{i}.mix.q.norm"])
    typed, tensors = make_model(cfg, seed=11, change=change)
    return cfg, typed, tensors


def sequence_with_mark(vocab, n, at, seed):
    from replay_cases import random_tokens
    toks = [t if t != MARK else (t + 1) % vocab for t in random_tokens(vocab, n, seed)]
    toks[at] = MARK
    return toks


def moves(cfg, tensors, toks, at, exact=None):
    """How far the logits of every position move when the token at `at` is another one, as a part of the largest logit."""
    exact = plain_tevovik_logits(cfg, tensors, toks) if exact is None else exact
    other = [t if i != at else (t + 2) % cfg["vocab"] for i, t in enumerate(toks)]
    return (plain_tevovik_logits(cfg, tensors, other) - exact).abs().max(dim=1).values / float(exact.abs().max())
