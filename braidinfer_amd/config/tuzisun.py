"""Typed configuration of the `Tuzisun` design and its translation into parts.

A Tuzisun model keeps its residual as `streams` rows a token, all equal to the embedding output at first and summed in
front of the final norm.  Each half of a layer reads one learnt weighted sum of the streams, normed by an element-wise
tanh(alpha x) w + b, and its output goes back into all of them through a learnt vector, beside a learnt mixing of the
streams themselves.  Mixers:

* `"parallel"`: two mixers side by side on the same input, their outputs summed with the weights `left_scale` and
  `right_scale`.  `left` is grouped-query attention in a sliding window of `mask.size` positions with biases on all four
  projections, an RMS norm per head of queries and keys and a rotation of the first `rot.dims` elements of every head in
  pairs of neighbours.  `right` is Mamba-2: `heads` of `vdim` channels over a state of `state` channels, `groups` of B
  and C, a convolution of `conv` taps, the gated output normed in `norm_groups` equal parts.
* `"mlstm"`: a matrix memory with exponential gates whose logarithms are bounded by `gate_cap`.
* `"channel_delta"`: a gated delta rule with a decay per head and key channel behind convolutions of `conv` taps; the
  decays and the sigmoid gate come through low-rank projections.

The feed-forward is a clamped gated unit, a set of routed experts (the softmax over all experts is the score, only experts
of the `groups.keep` runs of neighbours with the largest single scores can be chosen, the chosen scores are the weights as
they are) or absent.  The embedding table is the output head.  The reference has no such model; its configuration is one
flat struct (crates/braidinfer-runtime/src/config.rs:75-115), this one keeps the nesting of the design's config.json:

    {"architecture": "Tuzisun", "vocab": V, "width": W, "streams": s, "norm": {"eps": e},
     "layers": [{"type": "parallel",
                 "mixer": {"left": {"heads", "kv_heads", "dim", "vdim", "scale", "mask": {"size"}, "rot": {"base", "dims"}}, "left_scale",
                           "right": {"heads", "vdim", "state", "groups", "norm_groups", "conv"}, "right_scale"},
                 "mlp": {"kind": "dense", "ff": F, "limit": L}
                      | {"kind": "moe", "expert": {"ff": F}, "router": {"experts": E, "top": k, "groups": {"count", "keep"}}} | null},
                {"type": "mlstm", "mixer": {"heads", "dim", "vdim", "gate_cap"}, ...},
                {"type": "channel_delta", "mixer": {"heads", "kv_heads", "dim", "vdim", "conv", "decay_rank"?, "gate_rank"?}, ...}]}

`decay_rank` and `gate_rank` (the inner widths of a channel_delta layer's two low-rank projections) may be left out of
config.json: they are then read from the shapes of the layer's `mix.a1` and `mix.g1` tensors when the configuration comes
from a model folder.  Other keys that may be left out: `streams` (1), `left_scale`, `right_scale` (1), and in a mixer or
feed-forward `kv_heads` (as many as heads), `vdim` (dim), `mask` (every earlier token), `rot` (no rotation), `groups`,
`norm_groups` (1), `router.groups` (any expert can be chosen).

Tensor names: `embed`, `final.norm` (each norm: the weight, `.b` and `.alpha`), and under `l<i>.`: `norm1`, `norm2`, `hc1.*`,
`hc2.*` (`in`, `out`, `mix`), `mix.*` (`mix.left.*`, `mix.right.*` in a parallel layer), `mlp.gate|up|down` or
`mlp.e<j>.gate|up|down` and `mlp.router`.
"""
from __future__ import annotations

import copy
from dataclasses import dataclass, replace
from typing import Any, Callable, Dict, List, Optional, Tuple

from ..errors import ConfigError
from .kesitar import MAX_POSITIONS, _num, _pos_int
from .spec import LayerSpec, ModelSpec, PartSpec, ScheduleEntry

ARCHITECTURE = "Tuzisun"
MIXERS = ("parallel", "mlstm", "channel_delta")
GLU_ALPHA = 1.702          # the design's constant in g * sigmoid(alpha g)
RANKS = {"decay_rank": "a1", "gate_rank": "g1"}          # sizes of a channel_delta layer that only tensors may give


def _number(d, key: str, where: str, required: bool = True, default=None) -> float:
    return float(_num(d, key, where, kind=(int, float), required=required, default=default))


def _positive(d, key: str, where: str) -> float:
    v = _number(d, key, where)
    if not v > 0:
        raise ConfigError(f"config.json: {where}.{key} must be positive, found {v}")
    return v


def _check_multiple(m, where: str) -> None:
    heads = _pos_int(m, "heads", where)
    kv = _pos_int(m, "kv_heads", where, required=False, default=heads)
    if heads % kv:
        raise ConfigError(f"config.json: {where}: {heads} heads are not a multiple of {kv} key heads")


def _check_parallel(m, where: str) -> None:
    for side in ("left", "right"):
        if not isinstance(m.get(side), dict):
            raise ConfigError(f"config.json: {where}.{side} must be an object")
        _number(m, side + "_scale", where, required=False, default=1.0)
    a, at = m["left"], where + ".left"
    _check_multiple(a, at)
    dim = _pos_int(a, "dim", at)
    _pos_int(a, "vdim", at, required=False)
    _number(a, "scale", at)
    for key in ("mask", "rot"):
        if a.get(key) is not None and not isinstance(a[key], dict):
            raise ConfigError(f"config.json: {at}.{key} must be an object")
    if a.get("mask") is not None:
        _pos_int(a["mask"], "size", at + ".mask")
    if a.get("rot") is not None:
        dims = _pos_int(a["rot"], "dims", at + ".rot")
        if dims % 2 or dims > dim:
            raise ConfigError(f"config.json: {at}.rot.dims must be even and at most {dim}, found {dims}")
        _positive(a["rot"], "base", at + ".rot")
    s, at = m["right"], where + ".right"
    heads, vdim = _pos_int(s, "heads", at), _pos_int(s, "vdim", at)
    _pos_int(s, "state", at)
    _pos_int(s, "conv", at)
    groups = _pos_int(s, "groups", at, required=False, default=1)
    parts = _pos_int(s, "norm_groups", at, required=False, default=1)
    if heads % groups or (heads * vdim) % parts:
        raise ConfigError(f"config.json: {at}: {heads} heads of {vdim} channels do not divide into {groups} groups and {parts} normed parts")


def _check_mlp(mlp, where: str) -> None:
    if not isinstance(mlp, dict) or mlp.get("kind") not in ("dense", "moe"):
        raise ConfigError(f"config.json: {where}.kind must be 'dense' or 'moe', found {mlp!r}")
    if mlp["kind"] == "dense":
        _pos_int(mlp, "ff", where)
        _positive(mlp, "limit", where)
        return
    _pos_int(mlp.get("expert"), "ff", where + ".expert")
    n = _pos_int(mlp.get("router"), "experts", where + ".router")
    top = _pos_int(mlp["router"], "top", where + ".router")
    groups = mlp["router"].get("groups")
    count = keep = 1
    if groups is not None:
        count, keep = _pos_int(groups, "count", where + ".router.groups"), _pos_int(groups, "keep", where + ".router.groups")
    if n % count or keep > count or top > keep * (n // count):
        raise ConfigError(f"config.json: {where}.router chooses {top} of {n} experts within {keep} of {count} groups")


@dataclass(frozen=True)
class TuzisunConfig:
    vocab: int
    width: int
    streams: int
    norm_eps: float
    layers: Tuple[Dict[str, Any], ...]        # as in config.json, checked

    architecture = ARCHITECTURE

    @classmethod
    def from_dict(cls, d: Dict[str, Any]) -> "TuzisunConfig":
        layers = d.get("layers")
        if not isinstance(layers, (list, tuple)) or not layers:
            raise ConfigError("config.json: 'layers' must be a non-empty list")
        cfg = cls(vocab=_pos_int(d, "vocab", "the model"), width=_pos_int(d, "width", "the model"),
                  streams=_pos_int(d, "streams", "the model", required=False, default=1),
                  norm_eps=_number(d.get("norm"), "eps", "norm"), layers=tuple(copy.deepcopy(l) for l in layers))
        cfg.validate()
        return cfg

    # ---- sizes that only the tensors give -------------------------------------------------
    def missing_tensor_sizes(self) -> List[str]:
        """Names of the tensors whose shapes complete this configuration (`with_tensor_shapes`)."""
        return [f"l{i}.mix.{tensor}" for i, l in enumerate(self.layers) if l["type"] == "channel_delta"
                for key, tensor in RANKS.items() if l["mixer"].get(key) is None]

    def with_tensor_shapes(self, shape_of: Callable[[str], Optional[Tuple[int, ...]]]) -> "TuzisunConfig":
        """The configuration with every size config.json left to the tensors filled in; `shape_of(name)` is a
        tensor's shape or None."""
        layers = [copy.deepcopy(l) for l in self.layers]
        for name in self.missing_tensor_sizes():
            i, tensor = int(name[1:name.index(".")]), name.rsplit(".", 1)[1]
            key = next(k for k, t in RANKS.items() if t == tensor)
            shape = shape_of(name)
            if shape is None or len(shape) != 2 or shape[1] != self.width or shape[0] <= 0:
                raise ConfigError(f"config.json: layers[{i}].mixer has no '{key}' and the tensor {name} "
                                  f"({'absent' if shape is None else tuple(shape)}) does not give one")
            layers[i]["mixer"][key] = int(shape[0])
        return replace(self, layers=tuple(layers))

    def validate(self) -> None:
        if self.norm_eps < 0:
            raise ConfigError(f"config.json: norm.eps must not be negative, found {self.norm_eps}")
        for i, l in enumerate(self.layers):
            where = f"layers[{i}]"
            if not isinstance(l, dict) or l.get("type") not in MIXERS:
                raise ConfigError(f"config.json: {where}.type must be one of {MIXERS}, found {l.get('type') if isinstance(l, dict) else l!r}")
            m = l.get("mixer")
            if not isinstance(m, dict):
                raise ConfigError(f"config.json: {where} has no 'mixer'")
            at = where + ".mixer"
            if l["type"] == "parallel":
                _check_parallel(m, at)
            else:
                _check_multiple(m, at)
                _pos_int(m, "dim", at)
                _pos_int(m, "vdim", at, required=False)
                if l["type"] == "mlstm":
                    _positive(m, "gate_cap", at)
                else:
                    _pos_int(m, "conv", at)
                    for key in RANKS:
                        _pos_int(m, key, at, required=False)
            if l.get("mlp") is not None:
                _check_mlp(l["mlp"], f"layers[{i}].mlp")

    def to_dict(self) -> Dict[str, Any]:
        return {"architecture": ARCHITECTURE, "vocab": self.vocab, "width": self.width, "streams": self.streams,
                "norm": {"eps": self.norm_eps}, "layers": [copy.deepcopy(l) for l in self.layers]}


def _rope(rot: Dict[str, Any], positions: Dict[str, PartSpec]) -> str:
    """The name of the rotary encoding of these numbers; one part per distinct (dims, base)."""
    name = f"rope{rot['dims']}@{float(rot['base'])!r}"
    positions[name] = PartSpec("rope", {"rotary_dim": rot["dims"], "theta": float(rot["base"]), "pairing": "adjacent",
                                        "frequencies_from_float64": True})
    return name


def build_spec(cfg: TuzisunConfig) -> ModelSpec:
    """Tuzisun as parts: `hyper_connected` layers over `streams` residual streams with `dynamic_tanh` norms; in a parallel
    layer a `pooled_window_attention` as the layer's mixer and a `state_space` beside it; `matrix_memory`;
    `gated_delta_rule` with decays per key channel; `clamped_glu` or `routed_experts`."""
    W = cfg.width
    missing = cfg.missing_tensor_sizes()
    if missing:
        raise ConfigError(f"the configuration leaves sizes to the tensors {missing}; read it from a model folder or give "
                          f"{sorted(RANKS)}")
    norm = PartSpec("dynamic_tanh", {"size": W, "tensor": ""})
    layers: List[LayerSpec] = []
    positions: Dict[str, PartSpec] = {}
    for i, l in enumerate(cfg.layers):
        m, more, scales = l["mixer"], {}, [1.0]
        names = {"norm.mixer": "norm1"}
        if l["type"] == "parallel":
            a, s = m["left"], m["right"]
            scales = [float(m.get("left_scale", 1.0)), float(m.get("right_scale", 1.0))]
            rot = a.get("rot")
            mixer = PartSpec("pooled_window_attention", {
                "hidden_size": W, "num_heads": a["heads"], "num_kv_heads": a.get("kv_heads") or a["heads"], "key_dim": a["dim"],
                "value_dim": a.get("vdim") or a["dim"], "window": (a.get("mask") or {}).get("size"), "pool": 0, "scale": float(a["scale"]),
                "sink": False, "bias": True, "out_bias": True, "qk_norm_eps": cfg.norm_eps,
                "position": _rope(rot, positions) if rot is not None else None,
                "names": {"q": "q", "k": "k", "v": "v", "o": "o", "q_bias": "q.b", "k_bias": "k.b", "v_bias": "v.b", "o_bias": "o.b",
                          "q_norm": "q.norm", "k_norm": "k.norm"}})
            more["right"] = PartSpec("state_space", {
                "hidden_size": W, "num_heads": s["heads"], "value_dim": s["vdim"], "state_dim": s["state"], "groups": s.get("groups") or 1,
                "norm_groups": s.get("norm_groups") or 1, "taps": s["conv"], "norm_eps": cfg.norm_eps})
            names.update({"mixer": "mix.left.", "mixer.right": "mix.right."})
        elif l["type"] == "mlstm":
            mixer = PartSpec("matrix_memory", {"hidden_size": W, "num_heads": m["heads"], "key_dim": m["dim"],
                                               "value_dim": m.get("vdim") or m["dim"], "gate_cap": float(m["gate_cap"]), "norm_eps": cfg.norm_eps})
            names["mixer"] = "mix."
        else:
            mixer = PartSpec("gated_delta_rule", {
                "hidden_size": W, "num_heads": m["heads"], "num_key_heads": m.get("kv_heads") or m["heads"], "key_dim": m["dim"],
                "value_dim": m.get("vdim") or m["dim"], "taps": m["conv"], "norm_eps": cfg.norm_eps, "decay_rank": m["decay_rank"],
                "gate_rank": m["gate_rank"], "gate": "sigmoid"})
            names["mixer"] = "mix."
        names["connection.mixer"] = "hc1."
        norms = {"mixer": norm}
        connections = {"mixer": PartSpec("hyper_connection", {"hidden_size": W, "streams": cfg.streams, "branch_scales": scales})}
        mlp, ffn = l.get("mlp"), None
        if mlp is not None:
            if mlp["kind"] == "dense":
                ffn = PartSpec("clamped_glu", {"hidden_size": W, "intermediate_size": mlp["ff"], "limit": float(mlp["limit"]),
                                               "alpha": GLU_ALPHA, "bias": False})
            else:
                groups = mlp["router"].get("groups") or {}
                ffn = PartSpec("routed_experts", {
                    "hidden_size": W, "intermediate_size": mlp["expert"]["ff"], "num_experts": mlp["router"]["experts"],
                    "top": mlp["router"]["top"], "scoring": "softmax_all", "correction": False, "groups": groups.get("count", 1),
                    "groups_keep": groups.get("keep", 1)})
            norms["feed_forward"] = norm
            connections["feed_forward"] = PartSpec("hyper_connection", {"hidden_size": W, "streams": cfg.streams})
            names.update({"norm.feed_forward": "norm2", "feed_forward": "mlp.", "connection.feed_forward": "hc2."})
        layers.append(LayerSpec(prefix=f"l{i}.", mixer=mixer, feed_forward=ffn, norms=norms, block="hyper_connected", names=names,
                                more_mixers=more, connections=connections))
    # a parallel layer's attention has cache unit i; recurrent mixers keep state only
    schedule = [ScheduleEntry(layer=i, cache=i if l["type"] == "parallel" else None) for i, l in enumerate(cfg.layers)]
    return ModelSpec(
        architecture=ARCHITECTURE, hidden_size=W, vocab_size=cfg.vocab,
        embedding=PartSpec("embedding", {"vocab_size": cfg.vocab, "hidden_size": W, "scale": 1.0, "tensor": ""}),
        layers=layers, schedule=schedule, final_norm=norm,
        lm_head=PartSpec("lm_head", {"vocab_size": cfg.vocab, "hidden_size": W, "tied_to": "embed", "scale": 1.0}),
        positions=positions, max_position_embeddings=MAX_POSITIONS,
        embedding_prefix="embed", final_norm_prefix="final.norm", lm_head_prefix="head.",
        stop_token_ids=[], bos_token_id=None, streams=cfg.streams,
        optional_tensors=[f"l{i}.{n}" for i, l in enumerate(cfg.layers) if l.get("mlp") is None
                          for n in ("norm2", "norm2.b", "norm2.alpha", "hc2.in", "hc2.out", "hc2.mix")])


# ------------------------------------------------------------------ presets ---------
def _parallel(heads, kv_heads, dim, window, rot_dims, s_heads, s_vdim, state, groups, norm_groups, left_scale=0.7, right_scale=0.8, base=10000.0):
    return {"type": "parallel", "mixer": {
        "left": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "scale": dim ** -0.5, "mask": {"size": window},
                 "rot": {"base": base, "dims": rot_dims}}, "left_scale": left_scale,
        "right": {"heads": s_heads, "vdim": s_vdim, "state": state, "groups": groups, "norm_groups": norm_groups, "conv": 4},
        "right_scale": right_scale}}


def _mlstm(heads, dim, vdim, gate_cap=15.0):
    return {"type": "mlstm", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "gate_cap": gate_cap}}


def _channel_delta(heads, kv_heads, dim, vdim, rank):
    return {"type": "channel_delta", "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": 4, "decay_rank": rank,
                                               "gate_rank": rank}}


def _dense(ff, limit=7.0):
    return {"kind": "dense", "ff": ff, "limit": limit}


def _moe(ff, experts, top, count, keep):
    return {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top, "groups": {"count": count, "keep": keep}}}


def _with(layer, mlp):
    return dict(copy.deepcopy(layer), mlp=mlp)


def _stack(parallel, mlstm, delta, dense, moe):
    """Eight layers p m p d p m p d, a clamped unit behind the parallel layers, experts behind the others."""
    return [_with(l, dense if l is parallel else moe) for l in (parallel, mlstm, parallel, delta) * 2]


# Shapes without a model folder: a tiny one for tests and tools, and two of the size of a real model's layers.
PRESETS: Dict[str, Dict[str, Any]] = {
    "tuzisun-tiny": dict(vocab=320, width=96, streams=3, norm={"eps": 1e-6}, layers=[
        _with(_parallel(6, 2, 16, 40, 8, 4, 24, 16, 2, 2), _dense(80, 1.5)),
        _with(_mlstm(3, 16, 24), _moe(32, 6, 2, 3, 2)),
        _with(_channel_delta(4, 2, 16, 24, 12), _moe(32, 6, 2, 3, 2)),
        _with(_parallel(6, 2, 16, 40, 8, 4, 24, 16, 2, 2), None)]),
    "tuzisun-1b": dict(vocab=32768, width=2048, streams=2, norm={"eps": 1e-6}, layers=_stack(
        _parallel(16, 4, 128, 4096, 64, 32, 64, 128, 4, 4), _mlstm(16, 128, 128), _channel_delta(16, 16, 128, 128, 128),
        _dense(5632), _moe(1408, 16, 4, 4, 2))),
    "tuzisun-7b": dict(vocab=32768, width=4096, streams=2, norm={"eps": 1e-6}, layers=_stack(
        _parallel(32, 8, 128, 4096, 64, 64, 64, 128, 8, 8), _mlstm(32, 128, 128), _channel_delta(32, 32, 128, 128, 128),
        _dense(14336), _moe(1792, 32, 8, 8, 4))),
}


def preset(name: str, **overrides) -> TuzisunConfig:
    if name not in PRESETS:
        raise ConfigError(f"unknown preset {name!r}; known: {sorted(PRESETS)}")
    d = dict(copy.deepcopy(PRESETS[name]), architecture=ARCHITECTURE)
    d.update(overrides)
    return TuzisunConfig.from_dict(d)
