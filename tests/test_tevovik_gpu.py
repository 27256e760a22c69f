"""The Tevovik decoder in the engine against the plain decoder (plain_tevovik.py): the new kernels one by one, every
mechanism alone at many sizes, the replay regimes (whole prompts, decoding through the cache, portions down to two
tokens, mixed batches under a pool and slots that are used again), inputs made so that a chunk's edge, a far key, one map
taken for the other or another layer's cache shows in the logits, long decoding, and greedy generation through the
scheduler."""
from __future__ import annotations

import math

import pytest
import torch

from llm_rs_amd import Engine, StepEntry
from llm_rs_amd.engine.trace import TraceReplayer
from llm_rs_amd.kernels import kernels
from plain_tevovik import plain_difference, plain_norm, plain_positions, plain_route, plain_softmax, plain_tevovik_logits, plain_unit
from replay_cases import collect, live_token_need, mixed, portions, random_tokens, tail_decoded, whole
from tevovik_cases import (CONFIGS, PAGE_SIZE, allowed_error, attention, check_rows, config, make_folder, make_model, marked_model, moe, moves, one_layer,
                           reference, sequence_with_mark)

pytestmark = pytest.mark.gpu
DTYPES = ["float32", "bfloat16"]
TORCH = {"float32": torch.float32, "bfloat16": torch.bfloat16}


def replay(engine, steps):
    replayer = TraceReplayer.for_engine(engine)
    outputs = []
    for step in steps:
        out = replayer.step(step)
        outputs.append(None if out is None else torch.from_numpy(out.copy()))
    return collect(steps, outputs)


def engine_for(typed, tensors, dtype, page_size, tokens, max_requests=4):
    return Engine(typed, tensors, dtype=dtype, page_size=page_size, num_pages=max(-(-tokens // page_size), 1), max_requests=max_requests)


def run_regimes(cfg, typed, tensors, dtype, page_size, requests, regimes, allowed=None):
    exact = reference(cfg, tensors, requests)
    allowed = allowed if allowed is not None else allowed_error(dtype, cfg, tensors, requests, exact)
    for name, steps in regimes.items():
        eng = engine_for(typed, tensors, dtype, page_size, live_token_need(steps, 64))
        check_rows(replay(eng, steps), exact, requests, allowed, name)
        core = eng.cache.core
        assert core.slots_in_use() == 0 and all(core.pages_free(g) == core.pages_total(g) for g in range(core.n_groups)), name


def close(got, want, dtype, what="", tol=None):
    tol = tol if tol is not None else (3e-6 if dtype == torch.float32 else 1e-2)
    err = float((got.detach().cpu().double() - want.double()).abs().max())
    assert err <= tol * max(float(want.abs().max()), 1e-3), (what, err, float(want.abs().max()))


def rand(*shape, seed=0, scale=1.0):
    return torch.randn(*shape, generator=torch.Generator().manual_seed(seed), dtype=torch.float32) * scale


# ---- the kernels one by one, against the same operation in plain tensor code ---------------------------------------

@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("D", [1, 5, 46, 320, 1024, 1500, 4096, 5000, 8192, 9001])
def test_the_norm_on_the_way_into_the_stream(D, dtype):
    dt = TORCH[dtype]
    h, y, w = rand(7, D, seed=D) * 3.0, rand(7, D, seed=1), rand(D, seed=2) * 0.3
    want = h.double() + plain_norm(y.double(), w.double(), 1e-5)
    hd, yd = h.cuda(), y.cuda()
    x = torch.empty(7, D, dtype=dt, device="cuda") if dtype == "bfloat16" else None
    kernels().post_norm(hd, yd, (1.0 + w).cuda(), x, 1e-5)
    close(hd, want, torch.float32, "stream")
    assert float(yd.abs().max()) == 0.0
    if x is not None:
        assert torch.equal(x.cpu(), hd.cpu().to(dt))
    before, yd = hd.clone(), y.cuda()
    kernels().post_norm(hd, yd, None, x)
    assert torch.equal(hd, before) and float(yd.abs().max()) == 0.0 and (x is None or torch.equal(x.cpu(), hd.cpu().to(dt)))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("width", [1, 7, 46, 320, 2048])
def test_the_embedding_with_its_position_vector(width, dtype):
    table = rand(11, width, seed=width).to(TORCH[dtype])
    positions = torch.tensor([0, 1, 2, 700, 4095, 5], dtype=torch.int32)
    tokens = torch.tensor([3, 10, 0, 0, 7, 3], dtype=torch.int32)
    rates = torch.tensor([10000.0 ** (-2.0 * i / width) for i in range((width + 1) // 2)], dtype=torch.float64)
    out = torch.empty(6, width, device="cuda")
    both = torch.stack([rates.float(), (rates - rates.float().double()).float()])
    kernels().embed_rows(out, table.cuda(), tokens.cuda(), 1.3, waves=(positions.cuda(), both.cuda()))
    waves = torch.zeros(6, width, dtype=torch.float64)
    for t, p in enumerate(positions.tolist()):
        for c in range(width):
            waves[t, c] = (math.cos if c % 2 else math.sin)(p * 10000.0 ** (-(c - c % 2) / width))
    assert torch.equal(waves[:3], plain_positions(3, width))
    want = table.double()[tokens.long()] * 1.3 + waves
    assert float((out.cpu().double() - want).abs().max()) < 2e-6


@pytest.mark.parametrize("E,groups,keep,top", [(1, 1, 1, 1), (6, 3, 2, 3), (8, 4, 1, 2), (12, 2, 1, 4), (64, 8, 3, 6), (100, 20, 20, 100), (300, 100, 7, 9), (1000, 4, 2, 30)])
@pytest.mark.parametrize("score", ["softmax", "sigmoid"])
def test_the_router_with_groups(E, groups, keep, top, score):
    T = 37
    logits = rand(T, E, seed=E) * 2.0
    weights = torch.empty(T, E, device="cuda")
    kernels().route_topk(logits.cuda(), weights, top, False, score, groups=groups, keep_groups=keep)
    chosen, soft = plain_route(logits.double(), top, groups, keep)       # (sigmoid keeps the order of the logits, as softmax does)
    s = soft if score == "softmax" else 1.0 / (1.0 + torch.exp(-logits.double()))
    want = torch.zeros(T, E, dtype=torch.float64)
    for t in range(T):
        want[t, chosen[t]] = s[t, chosen[t]]
    close(weights, want, torch.float32, "weights")
    assert ((weights.cpu() > 0).sum(1) == top).all()
    renormalized = torch.empty(T, E, device="cuda")
    kernels().route_topk(logits.cuda(), renormalized, top, True, score, groups=groups, keep_groups=keep)
    close(renormalized, want / want.sum(1, keepdim=True), torch.float32, "renormalized")


def test_equal_groups_and_equal_experts_go_by_their_index():
    logits = torch.zeros(3, 8)
    logits[1, 5] = 1.0
    logits[2, [3, 6]] = 2.0
    weights = torch.empty(3, 8, device="cuda")
    kernels().route_topk(logits.cuda(), weights, 2, False, groups=4, keep_groups=1)
    assert [r.nonzero().flatten().tolist() for r in weights.cpu()] == [[0, 1], [4, 5], [2, 3]]


@pytest.mark.parametrize("dtype", DTYPES)
def test_the_gated_silu_activation(dtype):
    T, ff, E = 19, 6, 3
    sums, wts = rand(T, 2 * ff * E, seed=3) * 3.0, rand(T, E, seed=4).abs()
    g, u = sums[:, 0::2].double(), sums[:, 1::2].double()
    want = g / (1.0 + torch.exp(-g)) * u
    out = torch.empty(T, ff * E, dtype=TORCH[dtype], device="cuda")
    kernels().act_weight(out, sums.cuda(), None, ff * E, "swiglu")
    close(out, want, TORCH[dtype], "dense")
    kernels().act_weight(out, sums.cuda(), wts.cuda(), ff, "swiglu")
    close(out, want * wts.double().repeat_interleave(ff, dim=1), TORCH[dtype], "times the experts' weights")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("T", [3, 300])
@pytest.mark.parametrize("H,G,d,dv", [(3, 1, 5, 7), (4, 2, 16, 32), (2, 2, 32, 20), (4, 1, 64, 128), (2, 1, 96, 64)])
def test_two_maps_are_finished_into_one_row_of_keys(H, G, d, dv, T, dtype):
    dt = TORCH[dtype]
    page, pages = 8, 40
    sums = rand(T, (H + G) * 2 * d + G * dv + 1, seed=d)
    qw, kw = 1.0 + rand(d, seed=1) * 0.2, 1.0 + rand(d, seed=2) * 0.2
    slots = torch.randperm(page * pages, generator=torch.Generator().manual_seed(3))[:T].to(torch.int32)
    kc, vc = torch.zeros(pages, G, page, 2 * d, dtype=dt, device="cuda"), torch.zeros(pages, G, dv, page, dtype=dt, device="cuda")
    q = torch.empty(T, H * 2 * d, dtype=dt, device="cuda")
    kernels().qkv_finish(sums.cuda()[:, :-1], None, q, slots.cuda(), kc, vc, H, G, d, dv, page, pages, True, 1e-5, q_weight=qw.cuda(), k_weight=kw.cuda(), maps=2)
    s = sums.double()
    close(q, (plain_unit(s[:, :2 * H * d].view(T, 2 * H, d), 1e-5) * qw.double()).reshape(T, -1), dt, "q")
    k = (plain_unit(s[:, 2 * H * d:2 * (H + G) * d].reshape(T, 2 * G, d), 1e-5) * kw.double()).view(T, G, 2 * d)
    at, off = slots.long() // page, slots.long() % page
    close(kc.cpu()[at, :, off], k, dt, "keys")
    close(vc.cpu()[at, :, :, off], s[:, 2 * (H + G) * d:-1].reshape(T, G, dv), dt, "values")


def plain_expert_sum(x, t, weights, E, act, limit, alpha):
    """sum_e weights[:, e] Wdown_e act(..), from the part's tensors."""
    out = torch.zeros_like(x)
    for e in range(E):
        u = x @ t[f"x.experts.{e}.up_proj.weight"].double().T
        if act == "relu2":
            a = torch.clamp(u, min=0.0) ** 2
        else:
            g = x @ t[f"x.experts.{e}.gate_proj.weight"].double().T
            if act == "swiglu":
                a = g / (1.0 + torch.exp(-g)) * u
            else:
                g, u = torch.clamp(g, max=limit), torch.clamp(u, min=-limit, max=limit)
                a = g / (1.0 + torch.exp(-alpha * g)) * (u + 1.0)
        out += (a * weights[:, e:e + 1]) @ t[f"x.experts.{e}.down_proj.weight"].double().T
    return out


@pytest.mark.parametrize("act", ["swiglu", "clamped_glu", "relu2"])
@pytest.mark.parametrize("E,top,D,F", [(5, 2, 64, 64), (16, 4, 320, 128), (70, 3, 192, 64), (12, 1, 128, 192), (3, 2, 640, 320)])
def test_experts_over_their_own_rows(E, top, D, F, act):
    """The products over the rows that chose each expert (grouped tiles) and those of steps of few tokens that leave unchosen
    experts unread, at token counts around every kernel's bounds, against plain tensor code; an expert that nobody chose, one
    that everybody chose, weights of exactly zero."""
    k = kernels()
    g = torch.Generator().manual_seed(E + F)
    n_up = F if act == "relu2" else 2 * F
    up, down = (torch.randn(E, n_up, D, generator=g) * 0.1).to(torch.bfloat16), (torch.randn(E, D, F, generator=g) * 0.1).to(torch.bfloat16)
    t = {}
    for e in range(E):
        t[f"x.experts.{e}.up_proj.weight"] = up[e] if act == "relu2" else up[e][1::2]
        t[f"x.experts.{e}.gate_proj.weight"] = up[e][0::2]
        t[f"x.experts.{e}.down_proj.weight"] = down[e]
    assert k.grouped_experts_take(D, F, torch.bfloat16) and not k.grouped_experts_take(D + 8, F, torch.bfloat16) and not k.grouped_experts_take(D, F, torch.float32)
    w_up, w_down = up.reshape(E * n_up, D).cuda(), down.permute(1, 0, 2).reshape(D, E * F).contiguous().cuda()
    for T in (1, 3, 4, 5, 16, 17, 33, 64, 65, 130, 257, 400):
        x = torch.randn(T, D, generator=g).to(torch.bfloat16)
        weights = torch.zeros(T, E)
        choice = torch.rand(T, E, generator=g)
        choice[:, 0] = 2.0 if top > 1 else choice[:, 0]          # everybody's
        choice[:, E - 1] = -1.0                                   # nobody's
        weights.scatter_(1, choice.topk(top, dim=1).indices, 0.1 + torch.rand(T, top, generator=g))
        weights[T // 2] = 0.0
        h = torch.randn(T, D, generator=g)
        want = plain_expert_sum(x.double(), t, weights.double(), E, act, 1.5, 1.702)
        wd, xd = weights.cuda(), x.cuda()
        if T <= 64:
            hd = h.cuda()
            a = torch.full((T, E * F), float("nan"), dtype=torch.bfloat16, device="cuda")
            k.expert_few_up(a, xd, w_up, wd, F, act, 1.5, 1.702)
            k.expert_few_down(hd, a, w_down, wd)
            close(hd.cpu() - h, want, torch.bfloat16, f"few, {T} tokens")
        hd, rows = h.cuda(), T * top
        counts, row_of = torch.empty(E, dtype=torch.int32, device="cuda"), torch.empty(T, E, dtype=torch.int32, device="cuda")
        row_token, row_weight = torch.empty(rows, dtype=torch.int32, device="cuda"), torch.empty(rows, 1, device="cuda")
        k.route_counts(wd, counts)
        assert counts.tolist() == (weights > 0).sum(0).tolist()
        k.route_rows(wd, counts, row_token, row_weight, row_of)
        a, y = torch.empty(rows, F, dtype=torch.bfloat16, device="cuda"), torch.empty(rows, D, device="cuda")
        k.expert_up(a, xd, row_token, w_up, counts, row_weight, F, act, 1.5, 1.702)
        k.expert_down(y, a, w_down, counts)
        k.combine_rows(hd, y, row_of)
        close(hd.cpu() - h, want, torch.bfloat16, f"grouped, {T} tokens")


class Paged:
    """Random keys and values of several requests, in pages handed out in random order."""

    def __init__(self, lens, G, width, dv, dtype, page, seed=0):
        self.page, self.G, self.width, self.dv = page, G, width, dv
        self.k = [rand(n, G, width, seed=seed + 7 * i).to(dtype) for i, n in enumerate(lens)]
        self.v = [rand(n, G, dv, seed=seed + 7 * i + 1).to(dtype) for i, n in enumerate(lens)]
        per = [-(-n // page) for n in lens]
        self.pages = sum(per) + 2
        order = torch.randperm(self.pages, generator=torch.Generator().manual_seed(seed)).tolist()
        self.table = torch.zeros(len(lens), max(per) + 1, dtype=torch.int32)
        kc, vc = torch.zeros(self.pages, G, page, width, dtype=dtype), torch.zeros(self.pages, G, dv, page, dtype=dtype)
        for e, n in enumerate(lens):
            for i in range(per[e]):
                self.table[e, i] = order.pop()
            for j in range(n):
                kc[self.table[e, j // page], :, j % page] = self.k[e][j]
                vc[self.table[e, j // page], :, :, j % page] = self.v[e][j]
        self.kc, self.vc = kc.cuda(), vc.cuda()


def plain_paged_attention(q, k, v, pos, H, G, d, scale, chunk, difference):
    """One query [H, maps * d] at `pos` over keys [n, G, maps * d] and values [n, G, dv]."""
    maps = 1 if difference is None else 2
    lo = pos // chunk * chunk if chunk else 0
    out = []
    for h in range(H):
        g = h // (H // G)
        a = []
        for m in range(maps):
            p = plain_softmax((k[lo:pos + 1, g, m * d:(m + 1) * d] @ q[h, m * d:(m + 1) * d])[None] * scale)[0]
            a.append(p @ v[lo:pos + 1, g])
        out.append(a[0] if maps == 1 else plain_difference(a[0], a[1], difference[0], 1.0 - difference[2], difference[1]))
    return torch.stack(out)


SHAPES = [(3, 1, 5, 7, 16), (6, 3, 10, 6, 4), (4, 2, 16, 32, 16), (4, 4, 16, 16, 16), (4, 1, 32, 64, 16), (12, 2, 32, 64, 16), (16, 1, 32, 64, 16), (5, 1, 32, 32, 16),
          (6, 2, 48, 96, 16), (4, 2, 64, 128, 16), (8, 1, 64, 64, 16), (32, 1, 64, 128, 16), (4, 4, 96, 192, 16), (2, 1, 96, 96, 16), (4, 2, 128, 256, 16),
          (3, 3, 128, 128, 16), (4, 2, 20, 40, 16), (2, 1, 64, 128, 8), (2, 2, 100, 300, 16)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("chunk", [0, 1, 24, 100])
@pytest.mark.parametrize("H,G,d,dv,page", SHAPES)
def test_differential_attention_over_pages(H, G, d, dv, page, chunk, dtype):
    """Prompt portions of several sizes, from the start, from inside a chunk and across its edges, beside single tokens
    just before, at and after an edge; with a gate per head.  The single tokens once more by themselves."""
    dt = TORCH[dtype]
    scale, diff = 1.5 / math.sqrt(d), (0.45, 1e-5, 0.7)
    portions_ = [(0, 61), (90, 45), (23, 2), (250, 1), (99, 1), (100, 1), (119, 1), (120, 1), (7, 3), (0, 1)]      # (start, tokens)
    cache = Paged([a + n for a, n in portions_], G, 2 * d, dv, dt, page, seed=d)

    def run(which):
        counts = [portions_[e][1] for e in which]
        T = sum(counts)
        q = (rand(T, H * 2 * d, seed=dv + T)).to(dt)
        gate = rand(T, H, seed=5) * 2.0
        starts = torch.tensor([0] + torch.tensor(counts).cumsum(0).tolist(), dtype=torch.int32)
        pos = torch.cat([torch.arange(portions_[e][0], sum(portions_[e])) for e in which]).to(torch.int32)
        entry = torch.cat([torch.full((c,), i) for i, c in enumerate(counts)]).to(torch.int32)
        lens = torch.tensor([sum(portions_[e]) for e in which], dtype=torch.int32)
        n_single = sum(c == 1 for c in counts)
        k = kernels()
        need = k.attention_scratch_floats(len(which), 2 * H, max(2 * d, dv), int(lens.max()), G, n_single)
        scratch = torch.empty(max(need, 1), device="cuda")
        out = torch.full((T, H * dv), float("nan"), dtype=dt, device="cuda")
        k.attention(q.cuda(), out, cache.kc, cache.vc, cache.table[which].contiguous().cuda(), entry.cuda(), pos.cuda(), starts.cuda(), lens.cuda(), H, G, 2 * d,
                    page, cache.pages, 0, scale, scratch, int(lens.max()), n_single, int(lens[[c == 1 for c in counts]].sum()), value_dim=dv,
                    gate=gate.cuda(), gate_per=dv, mask_chunk=chunk, difference=diff)
        want = torch.stack([plain_paged_attention(q[t].double().view(H, 2 * d), cache.k[which[int(entry[t])]].double(), cache.v[which[int(entry[t])]].double(),
                                                  int(pos[t]), H, G, d, scale, chunk, diff) for t in range(T)])
        want = want / (1.0 + torch.exp(-gate.double()))[:, :, None]
        # (the difference over its root mean square enlarges what the two maps' roundings leave where they nearly cancel)
        close(out.view(T, H, dv), want, dt, f"{len(which)} entries", tol=3e-5 if dtype == "float32" else 2.5e-2)
    run(list(range(len(portions_))))
    run([3, 4, 5, 6, 7, 9])


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,G,d,page", [(3, 1, 20, 4), (4, 2, 64, 16), (8, 1, 128, 16), (4, 4, 32, 16)])
def test_a_mask_in_chunks_without_the_second_map(H, G, d, page, dtype):
    dt = TORCH[dtype]
    cache = Paged([200, 97, 96, 40], G, d, d, dt, page, seed=d)
    which, counts, first = [0, 1, 2, 3], [70, 1, 1, 40], [130, 96, 95, 0]
    T = sum(counts)
    q = rand(T, H * d, seed=d + 1).to(dt)
    pos = torch.cat([torch.arange(a, a + c) for a, c in zip(first, counts)]).to(torch.int32)
    entry = torch.cat([torch.full((c,), i) for i, c in enumerate(counts)]).to(torch.int32)
    starts = torch.tensor([0, 70, 71, 72, 112], dtype=torch.int32)
    lens = torch.tensor([200, 97, 96, 40], dtype=torch.int32)
    k = kernels()
    scratch = torch.empty(k.attention_scratch_floats(4, H, d, 200, G, 2), device="cuda")
    out = torch.empty(T, H * d, dtype=dt, device="cuda")
    k.attention(q.cuda(), out, cache.kc, cache.vc, cache.table.cuda(), entry.cuda(), pos.cuda(), starts.cuda(), lens.cuda(), H, G, d, page, cache.pages, 0,
                d ** -0.5, scratch, 200, 2, 97, mask_chunk=48)
    want = torch.stack([plain_paged_attention(q[t].double().view(H, d), cache.k[int(entry[t])].double(), cache.v[int(entry[t])].double(), int(pos[t]), H, G, d,
                                              d ** -0.5, 48, None) for t in range(T)])
    close(out.view(T, H, d), want, dt, tol=1e-5 if dtype == "float32" else 1e-2)


# ---- every mechanism alone ------------------------------------------------------------------------------------------

ALONE = {
    "any sizes": attention(6, 3, 5, 7, 11),
    "one head": attention(1, 1, 8, 8, 33, diff=0.1),
    "values as wide as both maps": attention(4, 2, 32, 64, 24),
    "values as wide as one map": attention(8, 2, 32, 32, 40, diff=0.7),
    "heads of 64": attention(2, 1, 64, 128, 17),
    "heads of 128": attention(2, 2, 128, 256, 70),
    "values wider than both": attention(2, 1, 16, 96, 16),
    "a chunk of one": attention(4, 2, 16, 32, 1),
    "a chunk longer than any sequence": attention(4, 1, 16, 32, 1000),
    "experts in groups": attention(2, 1, 8, 8, 16, mlp=moe(12, 3, 9, (4, 2))),
    "experts without groups": attention(2, 2, 8, 8, 16, mlp=moe(7, 2, 10)),
    "all experts chosen": attention(2, 1, 8, 16, 16, mlp=moe(6, 6, 8, (3, 3))),
    "one expert of the best group": attention(2, 1, 8, 16, 16, mlp=moe(16, 1, 8, (8, 1))),
}


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("which", list(ALONE))
def test_one_layer_of_each_kind(which, dtype):
    cfg = one_layer(ALONE[which], width=48 if "6" in which or "map" in which else 41)
    typed, tensors = make_model(cfg, seed=1, calm_router=dtype == "bfloat16")
    requests = {f"r{i}": random_tokens(cfg["vocab"], n, i) for i, n in enumerate([37, 1, 2, 70])}
    run_regimes(cfg, typed, tensors, dtype, 4 if "any" in which else 16, requests,
                {"whole": whole(requests), "decoded": tail_decoded(requests, tail=5), "token by token": tail_decoded(requests, tail=1000),
                 "portions": portions(requests, (2, 3, 30)), "mixed": mixed(requests, live=3, prefill_sizes=(3, 2, 9))})


# ---- whole models in every regime -----------------------------------------------------------------------------------

@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("which", list(CONFIGS))
def test_replay_regimes(which, dtype):
    cfg = CONFIGS[which]
    typed, tensors = make_model(cfg, seed=3, calm_router=dtype == "bfloat16")
    lengths = [1, 2, 23, 70, 131, 40, 17]          # more requests than slots: slots and pages are used again
    requests = {f"r{i}": random_tokens(cfg["vocab"], n, 10 + i) for i, n in enumerate(lengths)}
    run_regimes(cfg, typed, tensors, dtype, PAGE_SIZE[which], requests,
                {"whole": whole(requests), "decoded": tail_decoded(requests, tail=32), "portions": portions(requests),
                 "portions of two and three": portions(requests, (2, 3)), "mixed": mixed(requests, live=4),
                 "mixed, two live": mixed(requests, live=2, prefill_sizes=(2, 31, 4))})


@pytest.mark.parametrize("dtype", DTYPES)
def test_a_batch_of_unequal_requests_equals_each_alone(dtype):
    cfg = CONFIGS["odd"]
    typed, tensors = make_model(cfg, seed=5, calm_router=dtype == "bfloat16")
    requests = {"long": random_tokens(cfg["vocab"], 90, 1), "short": random_tokens(cfg["vocab"], 2, 2),
                "one": random_tokens(cfg["vocab"], 1, 3), "mid": random_tokens(cfg["vocab"], 33, 4)}
    eng = engine_for(typed, tensors, dtype, 4, 4 * 128)
    together = [{"step": 0, "entries": [{"id": r, "tokens": t, "want": list(range(len(t)))} for r, t in requests.items()], "end": list(requests)}]
    rows_together = replay(eng, together)
    rows_alone = replay(eng, whole(requests))        # the same engine: the slots and pages of the batch, used again
    exact = reference(cfg, tensors, requests)
    allowed = allowed_error(dtype, cfg, tensors, requests, exact)
    check_rows(rows_together, exact, requests, allowed, "together")
    check_rows(rows_alone, exact, requests, allowed, "alone")


# ---- inputs under which a fault shows -------------------------------------------------------------------------------

MARKED = {"any sizes": dict(heads=3, kv_heads=1, dim=5, vdim=7), "both maps' width": dict(heads=4, kv_heads=2, dim=32, vdim=64),
          "one map's width": dict(heads=4, kv_heads=1, dim=32, vdim=32), "heads of 64": dict(heads=2, kv_heads=2, dim=64, vdim=128)}


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("which", list(MARKED))
def test_a_marked_key_shows_in_its_chunk_and_nowhere_else(which, dtype):
    """The mark at a chunk's first and last place, at a page's, at the sequence's start and far back in a long chunk: it
    moves every later position of its chunk by far more than rounding does, and no position of the next chunk at all."""
    for chunk, length, places in ((40, 131, (0, 15, 39, 40, 47, 79, 80)), (250, 520, (0, 249, 250, 255, 256))):
        cfg, typed, tensors = marked_model(chunk=chunk, **MARKED[which])
        eng = engine_for(typed, tensors, dtype, 16, 576)
        for at in places:
            toks = sequence_with_mark(cfg["vocab"], length, at, seed=at)
            requests = {"m": toks}
            exact = reference(cfg, tensors, requests)
            moved = moves(cfg, tensors, toks, at, exact["m"])
            end = min(at // chunk * chunk + chunk, length)
            allowed = allowed_error(dtype, cfg, tensors, requests, exact)
            assert float(moved[at:end].min()) > 2.0 * allowed and float(moved[at:end].max()) > 0.05, (which, at, float(moved[at:end].min()), allowed)
            assert float(moved[end:].abs().sum()) == 0.0
            for name, steps in {"whole": whole(requests), "decoded": tail_decoded(requests, tail=length - max(at - 3, 1) if length < 200 else 40),
                                "portions": portions(requests, (at + 1, 2, 64, 3) if at else (2, 3, 64))}.items():
                check_rows(replay(eng, steps), exact, requests, allowed, f"mark at {at} of chunks of {chunk}, {name}")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("chunk,second", [(20, 75), (75, 20), (33, 33), (16, 500)])
def test_a_layer_that_reads_anothers_keys_through_its_own_chunk(chunk, second, dtype):
    """The second layer has no keys of its own: its queries find the marked key of the first layer wherever their own chunk,
    shorter or longer than the first layer's, still holds it, also when the first layer's chunk has long passed."""
    cfg, typed, tensors = marked_model(heads=4, kv_heads=2, dim=32, vdim=64, chunk=chunk, second_chunk=second)
    for at in (0, 19, 20, 74):
        toks = sequence_with_mark(cfg["vocab"], 160, at, seed=at)
        requests = {"m": toks, "other": random_tokens(cfg["vocab"], 30, 3)}
        exact = reference(cfg, tensors, requests)
        moved = moves(cfg, tensors, toks, at, exact["m"])
        end = min(at // second * second + second, 160)
        allowed = allowed_error(dtype, cfg, tensors, requests, exact)
        assert float(moved[at:end].min()) > 2.0 * allowed, (at, float(moved[at:end].min()), allowed)
        run_regimes(cfg, typed, tensors, dtype, 16, requests,
                    {"whole": whole(requests), "decoded": tail_decoded(requests, tail=60), "portions": portions(requests, (21, 2, 40, 3)),
                     "mixed": mixed(requests, live=2, prefill_sizes=(40, 2, 7))}, allowed)


@pytest.mark.parametrize("dtype", DTYPES)
def test_what_a_wrong_constant_would_do_is_far_outside_the_bound(dtype):
    """lambda's sign and its base, 1 - diff, the score's scale, the gate and the position vector each move the logits by
    far more than the engine is allowed to differ."""
    cfg = config(48, 61, [attention(4, 2, 32, 64, 40, diff=0.3), attention(4, 2, 32, 64, 64, diff=0.6, kv_from=0)])
    typed, tensors = make_model(cfg, seed=13)
    requests = {"a": random_tokens(61, 100, 1), "b": random_tokens(61, 3, 2)}
    exact = reference(cfg, tensors, requests)
    allowed = allowed_error(dtype, cfg, tensors, requests, exact)

    def moved(change_cfg=None, change=None):
        import copy
        c, t = copy.deepcopy(cfg), dict(tensors)
        if change_cfg:
            change_cfg(c)
        if change:
            change(t)
        return float((reference(c, t, requests)["a"] - exact["a"]).abs().max()) / float(exact["a"].abs().max())
    for d in (moved(lambda c: c["layers"][0]["mixer"].update(diff=0.6)), moved(lambda c: c["layers"][1]["mixer"].update(scale=c["layers"][1]["mixer"]["scale"] * 0.5)),
              moved(change=lambda t: t.update({"l0.mix.g": t["l0.mix.g"] * 0})), moved(lambda c: c["embedding"].update(scale=1.6)),
              moved(change=lambda t: t.update({"l1.mix.lq1": -t["l1.mix.lq1"] * 2, "l1.mix.lk2": t["l1.mix.lk2"] * 3}))):
        assert d > 1.5 * allowed, (d, allowed)
    run_regimes(cfg, typed, tensors, dtype, 16, requests, {"whole": whole(requests), "decoded": tail_decoded(requests, tail=40),
                                                           "portions": portions(requests, (2, 33, 3))}, allowed)


@pytest.mark.parametrize("dtype", DTYPES)
def test_pages_and_slots_used_again(dtype):
    cfg = CONFIGS["plain"]
    typed, tensors = make_model(cfg, seed=4, calm_router=dtype == "bfloat16")
    first, second = random_tokens(cfg["vocab"], 50, 1), random_tokens(cfg["vocab"], 30, 2)
    eng = Engine(typed, tensors, dtype=dtype, page_size=16, num_pages=4, max_requests=1)      # one slot, pages for one request
    exact = reference(cfg, tensors, {"first": first, "second": second})
    allowed = allowed_error(dtype, cfg, tensors, {"first": first, "second": second}, exact)
    for rid, toks in (("first", first), ("second", second), ("first", first)):
        slot = eng.open_request()
        assert slot == 0
        head = eng.step([StepEntry(slot, 0, toks[:20], list(range(20)))]).cpu().clone()
        tail = eng.step([StepEntry(slot, 20, toks[20:], list(range(len(toks) - 20)))]).cpu()
        eng.close_request(slot)
        got = torch.cat([head, tail]).double()
        err = float((got - exact[rid]).abs().max()) / float(exact[rid].abs().max())
        assert err <= allowed, (rid, err, allowed)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("which", ["odd", "wide"])
def test_long_decoding_with_recorded_steps(which, dtype):
    cfg = CONFIGS[which]
    typed, tensors = make_model(cfg, seed=6, calm_router=dtype == "bfloat16")
    requests = {"a": random_tokens(cfg["vocab"], 330, 1), "b": random_tokens(cfg["vocab"], 321, 2)}
    exact = reference(cfg, tensors, requests)
    allowed = allowed_error(dtype, cfg, tensors, requests, exact)
    steps = [{"step": 0, "entries": [{"id": r, "tokens": t[:9], "want": list(range(9))} for r, t in requests.items()], "end": []}]
    for i in range(9, 330):
        live = [r for r, t in requests.items() if i < len(t)]
        steps.append({"step": len(steps), "entries": [{"id": r, "tokens": [requests[r][i]], "want": [0]} for r in live],
                      "end": [r for r in live if i == len(requests[r]) - 1]})
    # (pages for what the longest chunks hold, not for all of the tokens)
    held = max(l["mixer"]["mask"]["size"] for l in cfg["layers"])
    ps = PAGE_SIZE[which]
    eng = Engine(typed, tensors, dtype=dtype, page_size=ps, num_pages=2 * (-(-held // ps) + 4), max_requests=4)
    check_rows(replay(eng, steps), exact, requests, allowed, "decoding")
    assert eng.runner.graph_replays > 100           # the single-token steps were recorded and replayed


@pytest.mark.parametrize("dtype", DTYPES)
def test_a_step_of_more_than_a_thousand_tokens(dtype):
    cfg = config(64, 40, [attention(2, 1, 32, 64, 300, mlp=moe(4, 2, 24, (2, 1))), attention(2, 1, 32, 64, 700, kv_from=0, mlp=moe(3, 1, 16)),
                          attention(2, 2, 16, 20, 64)])
    typed, tensors = make_model(cfg, seed=12, calm_router=dtype == "bfloat16")
    requests = {"a": random_tokens(40, 1100, 1), "b": random_tokens(40, 40, 2)}
    exact = reference(cfg, tensors, requests)
    allowed = allowed_error(dtype, cfg, tensors, requests, exact)
    cuts = {"a": 1031, "b": 5}
    steps = [{"step": 0, "entries": [{"id": r, "tokens": t[:cuts[r]], "want": list(range(cuts[r]))} for r, t in requests.items()], "end": []},
             {"step": 1, "entries": [{"id": r, "tokens": t[cuts[r]:], "want": list(range(len(t) - cuts[r]))} for r, t in requests.items()], "end": list(requests)}]
    eng = engine_for(typed, tensors, dtype, 16, 1280)
    check_rows(replay(eng, steps), exact, requests, allowed, "two steps")


# ---- configurations drawn at random -----------------------------------------------------------------------------------

def random_configuration(seed):
    import random
    r = random.Random(1000 + seed)
    width = r.choice([24, 40, 63, 96, 136])
    layers = []
    for i in range(r.randint(2, 6)):
        count = r.choice([1, 2, 4])
        keep, per = r.randint(1, count), r.randint(1, 4)
        mlp = r.choice([None, moe(count * per, r.randint(1, keep * per), r.randint(3, 40), (count, keep)), moe(r.randint(2, 9), 1, 8 * r.randint(1, 6))])
        own = [j for j, l in enumerate(layers) if l["mixer"].get("kv_from") is None]
        if own and r.random() < 0.5:
            j = r.choice(own)
            o = layers[j]["mixer"]
            kv, dim, vdim, kv_from = o["kv_heads"], o["dim"], o["vdim"], j
        else:
            kv, dim, kv_from = r.choice([1, 2, 3]), r.choice([4, 10, 16, 32, 48, 64, 128]), None
            vdim = r.choice([2 * dim, dim, 4 * r.randint(1, 10), r.randint(1, 30)])
        layers.append(attention(kv * r.choice([1, 2, 4]), kv, dim, vdim, r.choice([1, 5, 16, 31, 64, 90, 400]), scale=r.uniform(0.5, 2.5) * dim ** -0.5,
                                diff=r.uniform(0.05, 0.9), kv_from=kv_from, mlp=mlp))
    return config(width, r.randint(30, 200), layers, eps=r.choice([1e-5, 1e-6, 1e-3]), scale=r.uniform(0.5, 4.0))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("seed", range(10))
def test_configurations_drawn_at_random(seed, dtype):
    cfg = random_configuration(seed)
    typed, tensors = make_model(cfg, seed=seed, calm_router=dtype == "bfloat16")
    requests = {f"r{i}": random_tokens(cfg["vocab"], n, 70 + i) for i, n in enumerate([150, 3, 66, 1, 35])}
    run_regimes(cfg, typed, tensors, dtype, 16, requests,
                {"whole": whole(requests), "decoded": tail_decoded(requests, tail=36), "portions": portions(requests, (2, 70, 3, 33)),
                 "mixed": mixed(requests, live=3)})


# ---- generation through the scheduler --------------------------------------------------------------------------------

def plain_greedy(cfg, tensors, prompt, n):
    toks, margins = list(prompt), []
    for _ in range(n):
        row = plain_tevovik_logits(cfg, tensors, toks)[-1]
        top = torch.topk(row, 2).values
        margins.append(float(top[0] - top[1]) / float(row.abs().max()))
        toks.append(int(torch.argmax(row)))
    return toks[len(prompt):], margins


@pytest.mark.parametrize("which", ["odd", "plain"])
def test_greedy_generation_through_the_scheduler(which):
    cfg = CONFIGS[which]
    typed, tensors = make_model(cfg, seed=8)
    prompts = [random_tokens(cfg["vocab"], n, 20 + n) for n in (1, 5, 19, 40, 3, 27)]
    eng = Engine(typed, tensors, dtype="float32", page_size=PAGE_SIZE[which], num_pages=96, max_requests=3, max_batch_tokens=24)
    outs = eng.generate(prompts, max_new_tokens=12)
    for prompt, out in zip(prompts, outs):
        want, margins = plain_greedy(cfg, tensors, prompt, 12)
        out = list(out.tokens if hasattr(out, "tokens") else out)
        for i, (a, b) in enumerate(zip(out, want)):
            if a != b:
                assert margins[i] < 1e-4, (prompt, i, out, want)       # a tie within rounding may fall either way
                break


# ---- the programs, on a model folder ----------------------------------------------------------------------------------

def test_the_programs_on_a_model_folder(tmp_path):
    """A folder with config.json and model.safetensors through `bin/trace_run` (a mixed trace under a small pool, both
    dtypes) and through `bin/llm-rs complete` (greedy): the architecture is chosen by the file."""
    import json
    import os
    import subprocess
    import sys

    import numpy as np
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    cfg = CONFIGS["plain"]
    folder = make_folder(tmp_path, cfg, seed=11, calm_router=True)
    typed, tensors = make_model(cfg, seed=11, calm_router=True)
    requests = {f"r{i}": random_tokens(cfg["vocab"], n, 50 + i) for i, n in enumerate([33, 2, 90, 47, 18])}
    exact = reference(cfg, tensors, requests)
    steps = mixed(requests, live=3)
    text = "".join(json.dumps(s) + "\n" for s in steps)
    for dtype in DTYPES:
        out = tmp_path / f"out_{dtype}"
        p = subprocess.run([sys.executable, os.path.join(root, "bin", "trace_run"), "--model", folder, "--dtype", dtype, "--out", str(out),
                            "--max-tokens", str(live_token_need(steps, 64))], input=text, capture_output=True, text=True, timeout=600)
        assert p.returncode == 0, p.stderr[-2000:]
        assert [l for l in p.stdout.split("\n") if l.startswith("done")] == [f"done {s['step']}" for s in steps]
        outputs = []
        for s in steps:
            n = sum(len(e["want"]) for e in s["entries"])
            outputs.append(torch.from_numpy(np.fromfile(out / f"{s['step']}.f32", dtype="<f4").reshape(n, cfg["vocab"]).copy()) if n else None)
        check_rows(collect(steps, outputs), exact, requests, allowed_error(dtype, cfg, tensors, requests, exact), f"trace_run {dtype}")
    prompt = requests["r3"]
    p = subprocess.run([sys.executable, os.path.join(root, "bin", "llm-rs"), "-m", folder, "--dtype", "float32", "--num-pages", "64", "complete",
                        "--prompt-ids", " ".join(map(str, prompt)), "-n", "10", "--temperature", "0"], capture_output=True, text=True, timeout=600)
    assert p.returncode == 0, p.stderr[-2000:]
    got = [int(t) for t in p.stdout.split()]
    want, margins = plain_greedy(cfg, tensors, prompt, 10)
    for i, (a, b) in enumerate(zip(got, want)):
        if a != b:
            assert margins[i] < 1e-4, (i, got, want)
            break
    assert len(got) == 10
