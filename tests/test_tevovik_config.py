"""The Tevovik configuration, what the model asks of weights and cache, the plain decoder's own invariants, and the
engine's host logic on the emulated kernels (CPU)."""
from __future__ import annotations

import copy
import math

import pytest
import torch

from emulated_kernels import EmulatedKernels
from llm_rs_amd import ConfigError, Engine, Model, PagedKV, PartSpec, TevovikConfig, config_from_dict, load_config, use_kernels
from llm_rs_amd.engine.trace import TraceReplayer
from llm_rs_amd.parts.base import build_feed_forward, build_mixer
from plain_tevovik import (plain_attention, plain_chunk_mask, plain_difference, plain_embed, plain_expert, plain_experts, plain_lambda, plain_norm,
                           plain_positions, plain_route, plain_softmax, plain_tevovik_logits, plain_unit)
from replay_cases import collect, live_token_need, mixed, portions, random_tokens, tail_decoded, whole
from tevovik_cases import CONFIGS, PAGE_SIZE, attention, check_rows, config, make_folder, make_model, marked_model, moe, moves, one_layer, reference, sequence_with_mark

D = torch.float64


def test_the_registry_finds_the_architecture():
    cfg = config_from_dict(CONFIGS["odd"])
    assert isinstance(cfg, TevovikConfig) and cfg.to_dict() == CONFIGS["odd"]


@pytest.mark.parametrize("path", [("vocab",), ("width",), ("embedding", "scale"), ("norm", "eps"), ("layers", 0, "type"), ("layers", 0, "mixer", "heads"),
                                  ("layers", 0, "mixer", "dim"), ("layers", 0, "mixer", "vdim"), ("layers", 0, "mixer", "scale"), ("layers", 0, "mixer", "diff"),
                                  ("layers", 0, "mixer", "mask"), ("layers", 1, "mixer", "mask", "size"), ("layers", 0, "mlp", "kind"),
                                  ("layers", 0, "mlp", "expert", "ff"), ("layers", 0, "mlp", "router", "experts"), ("layers", 0, "mlp", "router", "top"),
                                  ("layers", 0, "mlp", "router", "groups", "keep"), ("layers", 0, "mlp", "router", "groups", "count")])
def test_a_missing_key_is_named(path):
    d = copy.deepcopy(CONFIGS["odd"])
    at = d
    for key in path[:-1]:
        at = at[key]
    del at[path[-1]]
    with pytest.raises(ConfigError, match=str(path[-1])):
        TevovikConfig.from_dict(d).model_spec()


def test_what_a_file_may_leave_out():
    d = copy.deepcopy(CONFIGS["odd"])
    del d["layers"][1]["mixer"]["kv_heads"], d["layers"][2]["mlp"]["router"]["groups"], d["layers"][1]["mlp"]
    spec = TevovikConfig.from_dict(d).model_spec()
    assert spec.layers[1].mixer.params["num_kv_heads"] == 3 and spec.layers[1].feed_forward is None
    assert spec.layers[2].feed_forward.params["groups"] == {"count": 1, "keep": 1}
    assert spec.ignorable_tensors == ("l1.norm2",)


def test_what_does_not_fit_is_refused():
    for change in (lambda d: d["layers"][0].update(type="mamba"), lambda d: d["layers"][0]["mixer"].update(kv_heads=4),
                   lambda d: d["layers"][0]["mlp"].update(kind="dense"), lambda d: d["layers"][0]["mixer"]["mask"].update(size=0),
                   lambda d: d["layers"][2]["mixer"].update(kv_from=2), lambda d: d["layers"][2]["mixer"].update(kv_from=5),
                   lambda d: d["layers"][3]["mixer"].update(kv_from=2), lambda d: d["layers"][2]["mixer"].update(dim=6),
                   lambda d: d["layers"][2]["mixer"].update(kv_heads=1), lambda d: d["layers"][2]["mixer"].update(vdim=7),
                   lambda d: d["layers"][0]["mlp"]["router"].update(top=5), lambda d: d["layers"][0]["mlp"]["router"].update(experts=7),
                   lambda d: d["layers"][0]["mlp"]["router"]["groups"].update(keep=4), lambda d: d["layers"][0]["mixer"].update(heads=0),
                   lambda d: d["norm"].update(eps=0.0), lambda d: d.update(layers=[])):
        d = copy.deepcopy(CONFIGS["odd"])
        change(d)
        with pytest.raises(ConfigError):
            TevovikConfig.from_dict(d).model_spec()


def test_who_reads_whose_cache_and_what_it_holds():
    spec = TevovikConfig.from_dict(CONFIGS["odd"]).model_spec()
    assert [r.cache_of for r in spec.schedule] == [None, None, 0, 0, None, 1]
    assert [layer.mixer.params["mask_chunk"] for layer in spec.layers] == [13, 50, 13, 29, 7, 10]
    # a cache holds what the largest chunk among the layers that look at it needs
    assert [layer.mixer.params["cache_window"] for layer in spec.layers] == [29, 50, 29, 29, 7, 50]
    assert [layer.mixer.params["kv_proj"] for layer in spec.layers] == [True, True, False, False, True, False]
    assert all(layer.block == "postnorm" and layer.mixer_norm is None for layer in spec.layers)
    assert spec.position_wave_base == 10000.0 and spec.embedding_scale == 1.7


def test_tensors_and_cache_needs():
    typed, tensors = make_model(CONFIGS["odd"], seed=1)
    model = Model(typed.model_spec(), torch.float32, "cpu")
    want = model.tensors()
    assert set(want) == set(tensors)
    assert want["l0.mix.q"].shape == (60, 45) and want["l0.mix.k"].shape == (20, 45) and want["l0.mix.v"].shape == (12, 45)
    assert want["l0.mix.o"].shape == (45, 36) and want["l0.mix.g"].shape == (6, 45) and want["l0.mix.lq1"].shape == (5,)
    assert want["l0.mix.q.norm"].shape == (5,) and "l2.mix.k" not in want and "l2.mix.k.norm" not in want and "l2.mix.v" not in want
    assert "l2.mix.lk2" in want and "l1.norm2" not in want and want["l0.mlp.e5.gate"].shape == (7, 45) and want["final.norm"].shape == (45,)
    needs = [need for need, _ in model.cache_needs()]
    assert needs[0] == needs[2] == needs[3] == PagedKV(2, 10, 29, 6) and needs[1] == needs[5] == PagedKV(3, 18, 50, 20) and needs[4] == PagedKV(1, 22, 7, 3)
    square = Model(TevovikConfig.from_dict(one_layer(attention(4, 2, 16, 32, 24))).model_spec(), torch.float32, "cpu")
    assert square.cache_needs()[0][0] == PagedKV(2, 32, 24)                     # values as wide as both maps' keys


def test_weights_come_back_as_the_file_had_them():
    for which in ("odd", "plain"):
        typed, tensors = make_model(CONFIGS[which], seed=2)
        model = Model(typed.model_spec(), torch.float32, "cpu")
        model.load(tensors)
        back = model.weights()
        assert set(back) == set(tensors)
        for name, t in tensors.items():
            assert torch.equal(back[name].float().reshape(t.shape), t.float()), name


def test_a_folder_is_read_by_its_architecture(tmp_path):
    folder = make_folder(tmp_path, CONFIGS["plain"], seed=3)
    assert isinstance(load_config(folder), TevovikConfig)


def test_options_that_do_not_go_together_are_refused():
    base = {"hidden_size": 16, "num_heads": 2, "num_kv_heads": 1, "head_dim": 4}
    for more in ({"mask_chunk": 8, "window": 4}, {"mask_chunk": -1}, {"difference": {"base": 0.5, "eps": 0.0}},
                 {"difference": {"base": 0.5, "eps": 1e-6}, "softcap": 3.0}, {"difference": {"base": 0.5, "eps": 1e-6}, "distance": "log"}):
        with pytest.raises(ValueError):
            build_mixer(PartSpec("attention", "x", {**base, **more}), torch.float32)
    ff = {"hidden_size": 16, "intermediate_size": 4, "experts": 6, "top": 2, "activation": "swiglu"}
    build_feed_forward(PartSpec("routed_ff", "x", {**ff, "groups": {"count": 3, "keep": 1}}), torch.float32)
    for groups in ({"count": 4, "keep": 1}, {"count": 3, "keep": 4}, {"count": 6, "keep": 1}):
        with pytest.raises(ValueError):
            build_feed_forward(PartSpec("routed_ff", "x", {**ff, "groups": groups}), torch.float32)


# ---- the plain decoder's mechanisms, worked out by hand ------------------------------------------------------------------

def test_plain_norm_is_around_one():
    x = torch.tensor([[3.0, 4.0]], dtype=D)
    r = math.sqrt(12.5 + 0.5)           # eps inside the root
    assert torch.allclose(plain_unit(x, 0.5), x / r) and torch.allclose(plain_norm(x, torch.tensor([0.0, -1.0], dtype=D), 0.5), torch.tensor([[3.0 / r, 0.0]], dtype=D))


def test_plain_positions_are_sines_and_cosines_side_by_side():
    p = plain_positions(4, 5)
    assert p[0].tolist() == [0.0, 1.0, 0.0, 1.0, 0.0]
    assert abs(float(p[3, 0]) - math.sin(3.0)) < 1e-12 and abs(float(p[3, 1]) - math.cos(3.0)) < 1e-12
    assert abs(float(p[2, 3]) - math.cos(2.0 * 10000.0 ** (-2.0 / 5.0))) < 1e-12 and abs(float(p[2, 4]) - math.sin(2.0 * 10000.0 ** (-4.0 / 5.0))) < 1e-12
    x = plain_embed(torch.tensor([[1.0, 2.0], [3.0, 4.0]], dtype=D), [1, 0], 2.0)
    assert torch.allclose(x, torch.tensor([[6.0, 9.0], [2.0 + math.sin(1.0), 4.0 + math.cos(1.0)]], dtype=D))


def test_plain_chunks_are_counted_from_the_start():
    m = plain_chunk_mask(7, 3, D)
    seen = [[j for j in range(7) if m[i, j] == 0.0] for i in range(7)]
    assert seen == [[0], [0, 1], [0, 1, 2], [3], [3, 4], [3, 4, 5], [6]]
    assert torch.equal(plain_chunk_mask(5, 100, D) == 0.0, torch.ones(5, 5, dtype=torch.bool).tril())
    assert torch.equal(plain_chunk_mask(4, 1, D) == 0.0, torch.eye(4, dtype=torch.bool))


def test_plain_lambda_and_difference():
    w = {"lq1": torch.tensor([1.0, 2.0], dtype=D), "lk1": torch.tensor([0.5, 0.25], dtype=D), "lq2": torch.tensor([-1.0, 0.0], dtype=D), "lk2": torch.tensor([2.0, 5.0], dtype=D)}
    lam = float(plain_lambda(w, 0.3))
    assert abs(lam - (math.exp(1.0) - math.exp(-2.0) + 0.3)) < 1e-12
    a1, a2 = torch.tensor([3.0, 1.0], dtype=D), torch.tensor([1.0, -1.0], dtype=D)
    o = plain_difference(a1, a2, 0.5, 0.25, 0.0)           # (2.5, 1.5), root mean square sqrt(4.25)
    assert torch.allclose(o, torch.tensor([2.5, 1.5], dtype=D) / math.sqrt(4.25) * 0.75)


def test_plain_attention_of_one_token_is_its_value_under_the_gate():
    cfg = one_layer(attention(2, 1, 3, 4, 5, diff=0.25), width=8, vocab=9)
    _, tensors = make_model(cfg, seed=5)
    w = {n[len("l0.mix."):]: t.double() for n, t in tensors.items() if n.startswith("l0.mix.")}
    m = cfg["layers"][0]["mixer"]
    h = torch.randn(1, 8, dtype=D, generator=torch.Generator().manual_seed(2))
    out, (k, v) = plain_attention(h, w, m, 1e-5)
    value = (w["v"] @ h[0]) * (1.0 - float(plain_lambda(w, 0.25)))              # both maps see this token alone
    o = value / torch.sqrt((value * value).mean() + 1e-5) * 0.75
    gates = 1.0 / (1.0 + torch.exp(-(w["g"] @ h[0])))
    assert torch.allclose(out[0], w["o"] @ torch.cat([o * gates[0], o * gates[1]]), atol=1e-12)
    assert torch.allclose(k[0, 0, 1], plain_unit((w["k"] @ h[0]).view(2, 3)[1], 1e-5) * w["k.norm"])
    # rows of k: map 1 first, then map 2; another layer's keys and values are used as they are
    other, _ = plain_attention(h, {**w, "k": w["k"] * 0.0, "v": w["v"] * 0.0}, m, 1e-5, (k, v))
    assert torch.allclose(other, out)


def test_plain_router_chooses_within_the_best_groups():
    z = torch.tensor([[5.0, -4.0, 3.0, 2.9, 1.0, 4.0]], dtype=D)
    s = plain_softmax(z)[0]
    for groups, keep, top, want in ((1, 1, 3, [0, 5, 2]), (3, 1, 2, [0, 1]), (3, 2, 3, [0, 5, 4]), (2, 1, 2, [0, 2]), (6, 6, 2, [0, 5])):
        chosen, scores = plain_route(z, top, groups, keep)
        assert chosen[0] == want, (groups, keep, chosen)
        assert torch.equal(scores[0], s)
    # (a group is as good as its best expert: the group of 5 and -4 beats the group of 3 and 2.9)


def test_plain_experts_are_weighed_by_their_scores_as_they_are():
    cfg = one_layer(attention(1, 1, 2, 2, 4, mlp=moe(4, 2, 3)), width=6, vocab=9)
    _, tensors = make_model(cfg, seed=4)
    w = {n[len("l0.mlp."):]: t.double() for n, t in tensors.items() if n.startswith("l0.mlp.")}
    h = torch.randn(5, 6, dtype=D, generator=torch.Generator().manual_seed(1))
    chosen, s = plain_route(h @ w["router"].T, 2, 1, 1)
    got = plain_experts(h, w, cfg["layers"][0]["mlp"])
    for t in range(5):
        want = sum(s[t, e] * plain_expert(h[t:t + 1], {k[3:]: v for k, v in w.items() if k.startswith(f"e{e}.")}, 1.0)[0] for e in chosen[t])
        assert torch.allclose(got[t], want, atol=1e-12)
    one = {"gate": torch.tensor([[2.0]], dtype=D), "up": torch.tensor([[3.0]], dtype=D), "down": torch.tensor([[1.0]], dtype=D)}
    assert abs(float(plain_expert(torch.tensor([[0.5]], dtype=D), one, 1.0)) - 1.0 / (1.0 + math.exp(-1.0)) * 1.5) < 1e-12


def test_the_sublayers_read_the_stream_and_their_results_are_normed():
    cfg = CONFIGS["odd"]
    _, tensors = make_model(cfg, seed=7)
    seen = []
    logits = plain_tevovik_logits(cfg, tensors, [3, 1, 4, 1, 5], after_layer=lambda i, x: seen.append(x.clone()))
    assert len(seen) == 6 and logits.shape == (5, 97)
    x = plain_embed(tensors["embed"].double(), [3, 1, 4, 1, 5], 1.7)
    w = {k[len("l0.mix."):]: t.double() for k, t in tensors.items() if k.startswith("l0.mix.")}
    ff = {k[len("l0.mlp."):]: t.double() for k, t in tensors.items() if k.startswith("l0.mlp.")}
    x = x + plain_norm(plain_attention(x, w, cfg["layers"][0]["mixer"], 1e-5)[0], tensors["l0.norm1"].double(), 1e-5)
    x = x + plain_norm(plain_experts(x, ff, cfg["layers"][0]["mlp"]), tensors["l0.norm2"].double(), 1e-5)
    assert torch.allclose(seen[0], x, atol=1e-12)


def test_marked_keys_show_inside_their_chunk_and_nowhere_else():
    cfg, _, tensors = marked_model(4, 2, 8, 12, 20)
    for at in (0, 19, 20, 33):
        moved = moves(cfg, tensors, sequence_with_mark(50, 70, at, seed=at), at)
        end = at // 20 * 20 + 20
        assert float(moved[at:end].min()) > 0.05 and float(moved[:at].abs().sum()) == 0.0 and float(moved[end:].abs().sum()) == 0.0


# ---- the engine's host logic on the emulated kernels ---------------------------------------------------------------

def replay_cpu(typed, tensors, dtype, page_size, steps, max_requests=4):
    with use_kernels(EmulatedKernels()):
        eng = Engine(typed, tensors, dtype=dtype, device="cpu", page_size=page_size, num_pages=max(-(-live_token_need(steps, 64) // page_size), 1),
                     max_requests=max_requests)
        rep = TraceReplayer.for_engine(eng)
        outputs = []
        for step in steps:
            out = rep.step(step)
            outputs.append(None if out is None else torch.from_numpy(out.copy()))
        core = eng.cache.core
        assert core.slots_in_use() == 0 and all(core.pages_free(g) == core.pages_total(g) for g in range(core.n_groups))
    return collect(steps, outputs)


@pytest.mark.parametrize("which", ["odd", "plain"])
def test_replay_regimes_on_the_host_logic(which):
    cfg = CONFIGS[which]
    typed, tensors = make_model(cfg, seed=3)
    lengths = [1, 2, 23, 50, 40, 17]            # more requests than slots: slots and pages are used again
    requests = {f"r{i}": random_tokens(cfg["vocab"], n, 10 + i) for i, n in enumerate(lengths)}
    exact = reference(cfg, tensors, requests)
    for name, steps in {"whole": whole(requests), "decoded": tail_decoded(requests, tail=12), "portions": portions(requests, (2, 3, 7)),
                        "mixed": mixed(requests, live=3)}.items():
        check_rows(replay_cpu(typed, tensors, "float32", PAGE_SIZE[which], steps), exact, requests, 3e-5, name)


def test_pages_that_no_chunk_can_see_go_back_and_a_readers_longer_chunk_keeps_them():
    for chunk, second, most in ((8, None, 8), (8, 24, 24)):
        cfg, typed, tensors = marked_model(2, 1, 4, 4, chunk, second)
        toks = sequence_with_mark(50, 60, 25, seed=1)
        with use_kernels(EmulatedKernels()):
            eng = Engine(typed, tensors, dtype="float32", device="cpu", page_size=4, num_pages=-(-most // 4) + 2, max_requests=1)
            rep = TraceReplayer.for_engine(eng)
            exact = reference(cfg, tensors, {"m": toks})["m"]
            for i in range(60):             # one token at a time, in a pool that holds little more than the longest chunk
                out = rep.step({"step": i, "entries": [{"id": "m", "tokens": [toks[i]], "want": [0]}], "end": ["m"] if i == 59 else []})
                err = float((torch.from_numpy(out.copy()).double()[0] - exact[i]).abs().max()) / float(exact.abs().max())
                assert err < 3e-5, (chunk, second, i, err)


def test_the_stack_takes_layers_of_other_arrangements():
    """A post-norm layer's hand-over to the next (its rows and the cleared room) is not taken for a norm of its own by a
    layer that norms first, and is made anew after one."""
    from llm_rs_amd.config.spec import LayerSpec, ModelSpec, RunSpec
    cfg = one_layer(attention(2, 1, 6, 8, 16, mlp=moe(3, 2, 5)), width=24)
    typed, tensors = make_model(cfg, seed=9)
    post = typed.model_spec().layers[0]
    norm = lambda name: PartSpec("rmsnorm", name, {"size": 24, "eps": 1e-5})
    pre = LayerSpec("prenorm", PartSpec("attention", "p.mix", {"hidden_size": 24, "num_heads": 2, "num_kv_heads": 1, "head_dim": 8, "position": None}),
                    PartSpec("swiglu", "p.ff", {"hidden_size": 24, "intermediate_size": 16}), norm("p.n1"), norm("p.n2"))
    spec = ModelSpec(24, 61, 1 << 20, [post, pre], [RunSpec(0), RunSpec(1), RunSpec(0), RunSpec(0)], norm("last"), "embed", None, position_wave_base=100.0)
    for dtype in (torch.float32, torch.bfloat16):
        model = Model(spec, dtype, "cpu")
        g = torch.Generator().manual_seed(3)
        own = {n: (tensors[n] if n in tensors and n != "embed" else torch.randn(t.shape, generator=g) * (0.3 if len(t.shape) > 1 else 0.1) + (1.0 if len(t.shape) == 1 else 0.0))
               for n, t in model.tensors().items()}
        outs = []
        for cut in (7, 3):
            with use_kernels(EmulatedKernels()):
                class Config:
                    def model_spec(self):
                        return spec
                eng = Engine(Config(), own, dtype=dtype, device="cpu", page_size=4, num_pages=16, max_requests=1)
                rep = TraceReplayer.for_engine(eng)
                toks = random_tokens(61, 7, 4)
                rows = [torch.from_numpy(rep.step({"entries": [{"id": "a", "tokens": part, "want": list(range(len(part)))}], "end": []}).copy())
                        for part in (toks[:cut], toks[cut:]) if part]
                outs.append(torch.cat(rows))
        assert torch.allclose(outs[0], outs[1], atol=1e-4 if dtype == torch.float32 else 5e-2) and torch.isfinite(outs[0]).all()
