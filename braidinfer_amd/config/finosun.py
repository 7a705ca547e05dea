"""Typed configuration of the `Finosun` design and its translation into parts.

A Finosun model is a stack of pre-norm layers whose halves are scaled channel by channel before they join the residual
rows: x += s1 * mixer(norm1(x)), then x += s2 * feed_forward(norm2(x)), with RMS norms of plain weights and learnt
vectors s1, s2.  A run of layers may be passed several times with the same weights (`loop`), every pass with caches of
its own; in front of every pass, the first one too, x <- W [x ; x0] with a learnt matrix and the embedding output x0.
Mixers:

* `"attention"`: grouped-query attention in a sliding window of `mask.size` positions; one RMS norm over the whole query
  (key) projection, rotation of the first `rot.dims` elements of every head in pairs of neighbours, every head's value
  divided by its root mean square, a learnt factor per head on its scores.
* `"latent_attention"`: keys and values of every head from one normed latent a token beside one rotated key part that
  all heads share (pairs i, i + rot.dims/2), queries projected directly, a sigmoid gate per output element.

The feed-forward is a set of routed experts or absent: the softmax over all router outputs is the score, a learnt
correction joins it for the choice only, the chosen scores are the weights as they are; the last outputs are identity
experts, which return their input; experts and the shared expert are clamped gated units, the shared one multiplied by
the sigmoid of one learnt product a token.  The embedding table is the output head.  The reference has no such model;
its configuration is one flat struct (crates/braidinfer-runtime/src/config.rs:75-115), this one keeps the nesting of
the design's config.json:

    {"architecture": "Finosun", "vocab": V, "width": W, "norm": {"eps": e}, "loop": {"start": a, "stop": b, "times": n},
     "layers": [{"type": "attention",
                 "mixer": {"heads", "kv_heads", "dim", "vdim", "scale", "mask": {"size"}, "rot": {"base", "dims"}},
                 "mlp": {"kind": "moe", "expert": {"ff": F, "limit": L}, "shared": {"ff": F, "limit": L},
                         "router": {"experts": E, "identity": I, "top": k}} | null},
                {"type": "latent_attention",
                 "mixer": {"heads", "dim", "rot_dim", "vdim", "kv_rank", "scale", "rot": {"base", "dims"}}, ...}]}

Keys that may be left out: `loop` (every layer once), `loop.times` (1), and in a mixer or feed-forward `kv_heads` (as
many as heads), `vdim` (dim), `mask` (every earlier token), `rot` (no rotation), `router.identity` (none), `shared`.
Tensor names: `embed`, `loop.in`, `final.norm`, and under `l<i>.`: `norm1`, `norm2`, `ls1`, `ls2`, `mix.*`,
`mlp.e<j>.gate|up|down`, `mlp.router`, `mlp.correction`, `mlp.shared.gate|up|down`, `mlp.shared.sg`.
"""
from __future__ import annotations

import copy
from dataclasses import dataclass
from typing import Any, Dict, List, Optional, Tuple

from ..errors import ConfigError
from .kesitar import MAX_POSITIONS, _num, _pos_int
from .spec import LayerSpec, ModelSpec, PartSpec, ScheduleEntry

ARCHITECTURE = "Finosun"
MIXERS = ("attention", "latent_attention")
GLU_ALPHA = 1.702          # the design's constant in g * sigmoid(alpha g)


def _positive(d, key: str, where: str) -> float:
    v = float(_num(d, key, where, kind=(int, float)))
    if not v > 0:
        raise ConfigError(f"config.json: {where}.{key} must be positive, found {v}")
    return v


def _check_rot(m, limit: int, where: str) -> None:
    rot = m.get("rot")
    if rot is None:
        return
    if not isinstance(rot, dict):
        raise ConfigError(f"config.json: {where}.rot must be an object")
    dims = _pos_int(rot, "dims", where + ".rot")
    if dims % 2 or dims > limit:
        raise ConfigError(f"config.json: {where}.rot.dims must be even and at most {limit}, found {dims}")
    _positive(rot, "base", where + ".rot")


@dataclass(frozen=True)
class FinosunConfig:
    vocab: int
    width: int
    norm_eps: float
    loop: Optional[Tuple[int, int, int]]      # (start, stop, times) or None
    layers: Tuple[Dict[str, Any], ...]        # as in config.json, checked

    architecture = ARCHITECTURE

    @classmethod
    def from_dict(cls, d: Dict[str, Any]) -> "FinosunConfig":
        layers = d.get("layers")
        if not isinstance(layers, (list, tuple)) or not layers:
            raise ConfigError("config.json: 'layers' must be a non-empty list")
        loop = d.get("loop")
        if loop is not None:
            loop = (int(_num(loop, "start", "loop", kind=int)), int(_num(loop, "stop", "loop", kind=int)),
                    int(_num(loop, "times", "loop", kind=int, required=False, default=1)))
        cfg = cls(vocab=_pos_int(d, "vocab", "the model"), width=_pos_int(d, "width", "the model"),
                  norm_eps=float(_num(d.get("norm"), "eps", "norm", kind=(int, float))), loop=loop,
                  layers=tuple(copy.deepcopy(l) for l in layers))
        cfg.validate()
        return cfg

    def validate(self) -> None:
        if self.norm_eps < 0:
            raise ConfigError(f"config.json: norm.eps must not be negative, found {self.norm_eps}")
        if self.loop is not None:
            start, stop, times = self.loop
            if not 0 <= start < stop <= len(self.layers) or times < 1:
                raise ConfigError(f"config.json: loop runs layers {start}..{stop - 1} {times} times; the model has "
                                  f"{len(self.layers)} layers")
        for i, l in enumerate(self.layers):
            where = f"layers[{i}]"
            if not isinstance(l, dict) or l.get("type") not in MIXERS:
                raise ConfigError(f"config.json: {where}.type must be one of {MIXERS}, found {l.get('type') if isinstance(l, dict) else l!r}")
            m = l.get("mixer")
            if not isinstance(m, dict):
                raise ConfigError(f"config.json: {where} has no 'mixer'")
            where += ".mixer"
            heads = _pos_int(m, "heads", where)
            dim = _pos_int(m, "dim", where)
            _pos_int(m, "vdim", where, required=False)
            _num(m, "scale", where, kind=(int, float))
            if l["type"] == "attention":
                kv = _pos_int(m, "kv_heads", where, required=False, default=heads)
                if heads % kv:
                    raise ConfigError(f"config.json: {where}: {heads} heads are not a multiple of {kv} kv heads")
                mask = m.get("mask")
                if mask is not None:
                    if not isinstance(mask, dict):
                        raise ConfigError(f"config.json: {where}.mask must be an object")
                    _pos_int(mask, "size", where + ".mask")
                _check_rot(m, dim, where)
            else:
                _pos_int(m, "kv_rank", where)
                rot_dim = _num(m, "rot_dim", where, kind=int)
                if rot_dim < 0:
                    raise ConfigError(f"config.json: {where}.rot_dim must not be negative, found {rot_dim}")
                if rot_dim:
                    _check_rot(m, rot_dim, where)
            mlp = l.get("mlp")
            if mlp is None:
                continue
            where = f"layers[{i}].mlp"
            if not isinstance(mlp, dict) or mlp.get("kind", "moe") != "moe":
                raise ConfigError(f"config.json: {where}.kind must be 'moe', found {mlp!r}")
            for key in ("expert", "shared"):
                if key == "expert" or mlp.get(key) is not None:
                    _pos_int(mlp.get(key), "ff", f"{where}.{key}")
                    _positive(mlp.get(key), "limit", f"{where}.{key}")
            n = _pos_int(mlp.get("router"), "experts", where + ".router")
            ident = _num(mlp["router"], "identity", where + ".router", kind=int, required=False, default=0)
            top = _pos_int(mlp["router"], "top", where + ".router")
            if ident < 0 or top > n + ident:
                raise ConfigError(f"config.json: {where}.router chooses {top} of {n} experts and {ident} identities")

    def to_dict(self) -> Dict[str, Any]:
        d = {"architecture": ARCHITECTURE, "vocab": self.vocab, "width": self.width, "norm": {"eps": self.norm_eps},
             "layers": [copy.deepcopy(l) for l in self.layers]}
        if self.loop is not None:
            d["loop"] = {"start": self.loop[0], "stop": self.loop[1], "times": self.loop[2]}
        return d

    def run_order(self) -> List[Tuple[int, bool]]:
        """(layer, whether the embedding output is joined in right before it) for every layer run, in order."""
        n = len(self.layers)
        if self.loop is None:
            return [(i, False) for i in range(n)]
        start, stop, times = self.loop
        order = [(i, False) for i in range(start)]
        for _ in range(times):
            order += [(i, i == start) for i in range(start, stop)]
        return order + [(i, False) for i in range(stop, n)]


def _rope(rot: Dict[str, Any], pairing: str, positions: Dict[str, PartSpec]) -> str:
    """The name of the rotary encoding of these numbers; one part per distinct (dims, base, pairing)."""
    name = f"rope{rot['dims']}@{float(rot['base'])!r}/{pairing}"
    positions[name] = PartSpec("rope", {"rotary_dim": rot["dims"], "theta": float(rot["base"]), "pairing": pairing,
                                        "frequencies_from_float64": True})
    return name


def build_spec(cfg: FinosunConfig) -> ModelSpec:
    """Finosun as parts: `sandwich_residual` layers with `rmsnorm` in front of the halves and `layer_scale` behind them; a
    `pooled_window_attention` with a norm over the projection, normed values and a factor a head, or a `latent_attention`
    with direct queries and a gate; `routed_experts` with scores over all outputs, identities and a gated shared unit; a
    `linear_join` in front of every pass; one run-order entry per layer run, each with a cache unit of its own."""
    W = cfg.width

    def norm():
        return PartSpec("rmsnorm", {"size": W, "eps": cfg.norm_eps, "tensor": ""})

    scale = PartSpec("layer_scale", {"size": W, "tensor": ""})
    layers: List[LayerSpec] = []
    positions: Dict[str, PartSpec] = {}
    for i, l in enumerate(cfg.layers):
        m = l["mixer"]
        rot = m.get("rot")
        if l["type"] == "attention":
            mixer = PartSpec("pooled_window_attention", {
                "hidden_size": W, "num_heads": m["heads"], "num_kv_heads": m.get("kv_heads", m["heads"]), "key_dim": m["dim"],
                "value_dim": m.get("vdim", m["dim"]), "window": (m.get("mask") or {}).get("size"), "pool": 0,
                "scale": float(m["scale"]), "sink": False, "bias": False, "qk_norm_eps": cfg.norm_eps,
                "qk_norm_over": "projection", "position": _rope(rot, "adjacent", positions) if rot is not None else None,
                "head_temp": True, "v_norm_eps": cfg.norm_eps,
                "names": {"q": "q", "k": "k", "v": "v", "o": "o", "q_norm": "q.norm", "k_norm": "k.norm", "head_temp": "temp"}})
        else:
            mixer = PartSpec("latent_attention", {
                "hidden_size": W, "num_heads": m["heads"], "head_dim": m["dim"], "rot_dim": m["rot_dim"],
                "value_dim": m.get("vdim", m["dim"]), "q_rank": None, "kv_rank": m["kv_rank"], "scale": float(m["scale"]),
                "norm_eps": cfg.norm_eps, "position": _rope(rot, "half", positions) if rot is not None and m["rot_dim"] else None,
                "sink": False, "gate": True})
        mlp, ffn = l.get("mlp"), None
        if mlp is not None:
            shared = mlp.get("shared") or {}
            ffn = PartSpec("routed_experts", {
                "hidden_size": W, "intermediate_size": mlp["expert"]["ff"], "num_experts": mlp["router"]["experts"],
                "top": mlp["router"]["top"], "scoring": "softmax_all", "identity": int(mlp["router"].get("identity", 0) or 0),
                "limit": float(mlp["expert"]["limit"]), "alpha": GLU_ALPHA, "shared_size": int(shared.get("ff", 0)),
                "shared_limit": float(shared["limit"]) if shared else None, "shared_gate": bool(shared)})
        norms = {"mixer": norm(), "mixer_out": scale}
        names = {"norm.mixer": "norm1", "norm.mixer_out": "ls1", "mixer": "mix."}
        if ffn is not None:
            norms.update({"feed_forward": norm(), "feed_forward_out": scale})
            names.update({"norm.feed_forward": "norm2", "norm.feed_forward_out": "ls2", "feed_forward": "mlp."})
        layers.append(LayerSpec(prefix=f"l{i}.", mixer=mixer, feed_forward=ffn, norms=norms, block="sandwich_residual", names=names))
    looped = cfg.loop is not None
    # every layer run has a cache unit of its own (a layer that is passed again shares weights, nothing else)
    schedule = [ScheduleEntry(layer=i, cache=n, input_join="pass" if joined else None) for n, (i, joined) in enumerate(cfg.run_order())]
    return ModelSpec(
        architecture=ARCHITECTURE, hidden_size=W, vocab_size=cfg.vocab,
        embedding=PartSpec("embedding", {"vocab_size": cfg.vocab, "hidden_size": W, "scale": 1.0, "tensor": ""}),
        layers=layers, schedule=schedule, final_norm=norm(),
        lm_head=PartSpec("lm_head", {"vocab_size": cfg.vocab, "hidden_size": W, "tied_to": "embed", "scale": 1.0}),
        positions=positions, max_position_embeddings=MAX_POSITIONS,
        embedding_prefix="embed", final_norm_prefix="final.norm", lm_head_prefix="head.",
        stop_token_ids=[], bos_token_id=None,
        input_joins={"pass": PartSpec("linear_join", {"hidden_size": W, "tensor": ""})} if looped else {},
        input_join_prefixes={"pass": "loop.in"} if looped else {},
        optional_tensors=[f"l{i}.{n}" for i, l in enumerate(cfg.layers) if l.get("mlp") is None for n in ("norm2", "ls2")])


# ------------------------------------------------------------------ presets ---------
def _attention(heads, kv_heads, dim, window, rot_dims, base=10000.0):
    return {"type": "attention", "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "scale": dim ** -0.5,
                                           "mask": {"size": window}, "rot": {"base": base, "dims": rot_dims}}}


def _latent(heads, dim, rot_dim, vdim, kv_rank, base=500000.0):
    return {"type": "latent_attention", "mixer": {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank,
                                                  "scale": (dim + rot_dim) ** -0.5, "rot": {"base": base, "dims": rot_dim}}}


def _moe(ff, experts, identity, top, shared, limit=7.0):
    return {"kind": "moe", "expert": {"ff": ff, "limit": limit}, "shared": {"ff": shared, "limit": limit},
            "router": {"experts": experts, "identity": identity, "top": top}}


def _with(layer, mlp):
    return dict(copy.deepcopy(layer), mlp=mlp)


# Shapes without a model folder: a tiny one for tests and tools, and two of the size of a real model's layers (eight
# layer runs each: a window layer, a latent and a window layer passed three times, a window layer).
PRESETS: Dict[str, Dict[str, Any]] = {
    "finosun-tiny": dict(vocab=320, width=96, norm={"eps": 1e-6}, loop={"start": 1, "stop": 3, "times": 2}, layers=[
        _with(_attention(6, 2, 16, 40, 8), _moe(32, 6, 2, 3, 48)),
        _with(_latent(3, 24, 8, 16, 40), _moe(32, 6, 2, 3, 48)),
        _with(_attention(6, 2, 16, 40, 8), None),
        _with(_latent(3, 24, 8, 16, 40), _moe(32, 6, 2, 3, 48))]),
    "finosun-1b": dict(vocab=32768, width=2048, norm={"eps": 1e-6}, loop={"start": 1, "stop": 3, "times": 3}, layers=[
        _with(_attention(16, 4, 128, 4096, 64), _moe(1408, 16, 4, 3, 1408)),
        _with(_latent(16, 64, 32, 64, 160), _moe(1408, 16, 4, 3, 1408)),
        _with(_attention(16, 4, 128, 4096, 64), _moe(1408, 16, 4, 3, 1408)),
        _with(_attention(16, 4, 128, 4096, 64), _moe(1408, 16, 4, 3, 1408))]),
    "finosun-7b": dict(vocab=32768, width=4096, norm={"eps": 1e-6}, loop={"start": 1, "stop": 3, "times": 3}, layers=[
        _with(_attention(32, 8, 128, 4096, 64), _moe(1792, 32, 8, 7, 1792)),
        _with(_latent(32, 64, 32, 64, 224), _moe(1792, 32, 8, 7, 1792)),
        _with(_attention(32, 8, 128, 4096, 64), _moe(1792, 32, 8, 7, 1792)),
        _with(_attention(32, 8, 128, 4096, 64), _moe(1792, 32, 8, 7, 1792))]),
}


def preset(name: str, **overrides) -> FinosunConfig:
    if name not in PRESETS:
        raise ConfigError(f"unknown preset {name!r}; known: {sorted(PRESETS)}")
    d = dict(copy.deepcopy(PRESETS[name]), architecture=ARCHITECTURE)
    d.update(overrides)
    return FinosunConfig.from_dict(d)
