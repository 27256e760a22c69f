"""Typed configuration of the Tevovik decoder, read from config.json.

A decoder whose layers are listed one by one.  The token table's rows times a constant, plus a vector of sines and cosines
of the position, enter the stream.  Both sublayers of a layer read the stream itself; their results are RMS-normed (the
weight stored as its distance from one) on the way back: x <- x + norm1(mixer(x)), x <- x + norm2(ff(x)).  The mixer is
differential attention: a head has two maps, each a softmax attention with queries and keys of its own (RMS-normed per head
and map, not rotated) over values that both share; the second map's result is taken off the first's lambda times, the
difference is RMS-normed over the head and multiplied by 1 - diff and by a sigmoid gate per head.  A query sees the keys of
its own chunk of `mask.size` positions, counted from the sequence's start.  A layer with `kv_from` j has no keys and values
of its own: its queries look at layer j's, through its own mask.  The feed-forward, where a layer has one, is a mixture of
gated (silu) experts: scores softmax(Wrouter x), the `top` experts with the largest scores among those of the best `keep` of
`count` groups, weighed by their scores as they are.  Final norm, an output matrix of its own.  Every size and every
constant that the file gives is read here.

config.json keys: architecture ("Tevovik"), vocab, width, embedding.scale, norm.eps and
layers[i] = {type: "attention", mixer: {...}, mlp: null | {...}} with
  mixer: heads, kv_heads (absent: heads), dim, vdim, scale, diff, mask.size, kv_from (absent: none)
  mlp:   {kind: "moe", expert: {ff}, router: {experts, top, groups (absent or null: one): {count, keep}}}
Tensors: embed, head, final.norm, and for layer i under "l<i>.": norm1, norm2 (with a feed-forward),
mix.{q, k, v, q.norm, k.norm, lq1, lk1, lq2, lk2, g, o} (k, v and k.norm not with kv_from), mlp.router,
mlp.e<j>.{gate, up, down}.
"""
from __future__ import annotations

import copy
from typing import Any, Dict, List

from .llama import ConfigError
from .spec import ExtraPart, LayerSpec, ModelSpec, PartSpec, RunSpec

MIXER_TYPES = ("attention",)
FF_KINDS = ("moe",)
WAVE_BASE = 10000.0         # of the position vector: the design fixes it
# The file gives no longest sequence: positions enter through sines, cosines and chunks only.
UNBOUNDED_POSITIONS = 1 << 24


def _need(d: Dict[str, Any], key: str, where: str):
    if not isinstance(d, dict) or d.get(key) is None:
        raise ConfigError(f"missing config key: {where}{key}")
    return d[key]


def _positive(d: Dict[str, Any], keys, where: str) -> None:
    for key in keys:
        if not int(_need(d, key, where)) > 0:
            raise ConfigError(f"{where}{key} must be positive, got {d[key]}")


class TevovikConfig:
    architecture = "Tevovik"

    def __init__(self, d: Dict[str, Any]):
        self.raw = copy.deepcopy(d)
        self.vocab = int(_need(d, "vocab", ""))
        self.width = int(_need(d, "width", ""))
        self.embedding_scale = float(_need(_need(d, "embedding", ""), "scale", "embedding."))
        self.eps = float(_need(_need(d, "norm", ""), "eps", "norm."))
        self.layers: List[Dict[str, Any]] = copy.deepcopy(list(_need(d, "layers", "")))
        for layer in self.layers:           # what a file may leave out: as many key heads as heads
            m = layer.get("mixer") if isinstance(layer, dict) else None
            if isinstance(m, dict) and m.get("kv_heads") is None and m.get("heads") is not None:
                m["kv_heads"] = m["heads"]
        self.validate()

    @classmethod
    def from_dict(cls, d: Dict[str, Any]) -> "TevovikConfig":
        return cls(d)

    def validate(self) -> None:
        if self.vocab <= 0 or self.width <= 0:
            raise ConfigError("vocab and width must be positive")
        if not self.eps > 0:
            raise ConfigError(f"norm.eps must be positive, got {self.eps}")
        if not self.layers:
            raise ConfigError("layers is empty")
        for i, layer in enumerate(self.layers):
            where = f"layers[{i}]."
            kind = _need(layer, "type", where)
            if kind not in MIXER_TYPES:
                raise ConfigError(f"{where}type: unknown mixer {kind!r} (known: {', '.join(MIXER_TYPES)})")
            m = _need(layer, "mixer", where)
            mw = where + "mixer."
            _positive(m, ("heads", "kv_heads", "dim", "vdim"), mw)
            for key in ("scale", "diff"):
                _need(m, key, mw)
            _positive(_need(m, "mask", mw), ("size",), mw + "mask.")
            if int(m["heads"]) % int(m["kv_heads"]):
                raise ConfigError(f"{mw}: {m['heads']} heads are no multiple of {m['kv_heads']} kv_heads")
            if m.get("kv_from") is not None:
                j = int(m["kv_from"])
                if not 0 <= j < i:
                    raise ConfigError(f"{mw}kv_from = {j}: not a layer before this one")
                other = self.layers[j]["mixer"]
                if other.get("kv_from") is not None:
                    raise ConfigError(f"{mw}kv_from = {j}: that layer has no keys and values of its own")
                for key in ("kv_heads", "dim", "vdim"):
                    if int(other[key]) != int(m[key]):
                        raise ConfigError(f"{mw}{key} = {m[key]}, but the keys and values of layer {j} were made with {other[key]}")
            mlp = layer.get("mlp")
            if mlp is not None:
                lw = where + "mlp."
                if _need(mlp, "kind", lw) not in FF_KINDS:
                    raise ConfigError(f"{lw}kind: unknown feed-forward {mlp['kind']!r} (known: {', '.join(FF_KINDS)})")
                _positive(_need(mlp, "expert", lw), ("ff",), lw + "expert.")
                r = _need(mlp, "router", lw)
                rw = lw + "router."
                _positive(r, ("experts", "top"), rw)
                count, keep = self._groups(r, rw)
                experts, top = int(r["experts"]), int(r["top"])
                if experts % count or keep > count:
                    raise ConfigError(f"{rw}groups: {experts} experts in {count} groups of which {keep} are kept")
                if top > experts // count * keep:
                    raise ConfigError(f"{rw}top = {top} of {experts // count * keep} experts")

    @staticmethod
    def _groups(router: Dict[str, Any], where: str):
        groups = router.get("groups")
        if groups is None:
            return 1, 1
        _positive(groups, ("count", "keep"), where + "groups.")
        return int(groups["count"]), int(groups["keep"])

    def to_dict(self) -> Dict[str, Any]:
        d = copy.deepcopy(self.raw)
        d["layers"] = copy.deepcopy(self.layers)
        return d

    # -- what the engine builds from -----------------------------------------------------------------------------
    def _held(self, i: int) -> int:
        """How many of a request's latest positions the cache that layer i writes or reads has to hold: the largest
        chunk among the layers that look at it."""
        source = self._source(i)
        return max(int(layer["mixer"]["mask"]["size"]) for j, layer in enumerate(self.layers) if self._source(j) == source)

    def _source(self, i: int) -> int:
        kv_from = self.layers[i]["mixer"].get("kv_from")
        return i if kv_from is None else int(kv_from)

    def _mixer(self, i: int, m: Dict[str, Any]) -> PartSpec:
        names = {"q": "q", "k": "k", "v": "v", "o": "o", "q_norm": "q.norm", "k_norm": "k.norm", "gate": "g"}
        return PartSpec("attention", f"l{i}.mix", {
            "hidden_size": self.width, "num_heads": int(m["heads"]), "num_kv_heads": int(m["kv_heads"]), "head_dim": int(m["dim"]),
            "value_dim": int(m["vdim"]), "position": None, "scale": float(m["scale"]), "qk_norm_eps": self.eps, "qk_norm_weight": True,
            "difference": {"base": float(m["diff"]), "eps": self.eps}, "mask_chunk": int(m["mask"]["size"]), "cache_window": self._held(i),
            "kv_proj": m.get("kv_from") is None, "gate": "head", "names": names})

    def _feed_forward(self, i: int, mlp: Dict[str, Any]) -> PartSpec:
        r = mlp["router"]
        count, keep = self._groups(r, "")
        return PartSpec("routed_ff", f"l{i}.mlp", {
            "hidden_size": self.width, "intermediate_size": int(mlp["expert"]["ff"]), "experts": int(r["experts"]), "top": int(r["top"]),
            "activation": "swiglu", "renormalize": False, "groups": {"count": count, "keep": keep},
            "names": {"router": "router", "expert": "e{}", "gate": "gate", "up": "up", "down": "down"}})

    def model_spec(self) -> ModelSpec:
        norm = lambda name: PartSpec("rmsnorm", name, {"size": self.width, "eps": self.eps, "tensor": "", "around_one": True})
        layers, schedule = [], []
        unused = []         # a layer without a feed-forward reads no second norm, whether or not its file holds one
        for i, layer in enumerate(self.layers):
            extra = [ExtraPart("post_mixer_norm", "norm", norm(f"l{i}.norm1"))]
            ff = None
            if layer.get("mlp") is None:
                unused.append(f"l{i}.norm2")
            else:
                ff = self._feed_forward(i, layer["mlp"])
                extra.append(ExtraPart("post_feed_forward_norm", "norm", norm(f"l{i}.norm2")))
            layers.append(LayerSpec("postnorm", self._mixer(i, layer["mixer"]), ff, None, None, tuple(extra)))
            kv_from = layer["mixer"].get("kv_from")
            schedule.append(RunSpec(i, cache_of=None if kv_from is None else int(kv_from)))
        return ModelSpec(hidden_size=self.width, vocab_size=self.vocab, max_positions=UNBOUNDED_POSITIONS, layers=layers,
                         schedule=schedule, final_norm=norm("final.norm"), embedding_name="embed", head_name="head",
                         embedding_scale=self.embedding_scale, position_wave_base=WAVE_BASE, ignorable_tensors=tuple(unused))
