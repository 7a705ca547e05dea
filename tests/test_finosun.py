"""The Finosun design on the host: configuration, run order and parts, tensor names, what the cache keeps, and the
plain implementation's mechanisms against direct sums."""
import copy
import math

import numpy as np
import pytest

import plain_finosun as P


def tiny():
    return {"architecture": "Finosun", "vocab": 90, "width": 40, "norm": {"eps": 1e-4}, "loop": {"start": 1, "stop": 3, "times": 2}, "layers": [
        {"type": "attention", "mixer": {"heads": 4, "kv_heads": 2, "dim": 8, "vdim": 12, "scale": 0.3, "mask": {"size": 9}, "rot": {"base": 100.0, "dims": 4}},
         "mlp": {"kind": "moe", "expert": {"ff": 16, "limit": 0.8}, "shared": {"ff": 24, "limit": 1.1}, "router": {"experts": 3, "identity": 2, "top": 2}}},
        {"type": "latent_attention", "mixer": {"heads": 3, "dim": 6, "rot_dim": 4, "vdim": 10, "kv_rank": 14, "scale": 0.4, "rot": {"base": 50.0, "dims": 4}},
         "mlp": None},
        {"type": "attention", "mixer": {"heads": 3, "kv_heads": 3, "dim": 6, "vdim": 6, "scale": 0.5, "mask": {"size": 5}, "rot": {"base": 30.0, "dims": 6}},
         "mlp": {"kind": "moe", "expert": {"ff": 12, "limit": 2.0}, "shared": {"ff": 12, "limit": 2.0}, "router": {"experts": 4, "identity": 1, "top": 3}}}]}


def test_configuration_is_read_and_checked():
    import braidinfer_amd as B
    from braidinfer_amd.errors import ConfigError
    cfg = B.config_from_dict(tiny())
    assert type(cfg).__name__ == "FinosunConfig" and cfg.loop == (1, 3, 2)
    assert B.config_from_dict(cfg.to_dict()) == cfg

    def broken(change):
        d = tiny()
        change(d)
        with pytest.raises(ConfigError):
            B.config_from_dict(d)
    broken(lambda d: d["layers"][0].__setitem__("type", "retention"))
    broken(lambda d: d["layers"][0]["mixer"].__setitem__("kv_heads", 3))
    broken(lambda d: d["layers"][0]["mixer"].__setitem__("mask", {"size": 0}))
    broken(lambda d: d["layers"][0]["mixer"]["rot"].__setitem__("dims", 3))
    broken(lambda d: d["layers"][0]["mixer"]["rot"].__setitem__("dims", 10))
    broken(lambda d: d["layers"][0]["mixer"].pop("scale"))
    broken(lambda d: d["layers"][1]["mixer"].pop("kv_rank"))
    broken(lambda d: d["layers"][1]["mixer"].__setitem__("rot_dim", -2))
    broken(lambda d: d["layers"][1]["mixer"]["rot"].__setitem__("dims", 6))
    broken(lambda d: d["layers"][0]["mlp"].__setitem__("kind", "dense"))
    broken(lambda d: d["layers"][0]["mlp"]["expert"].pop("limit"))
    broken(lambda d: d["layers"][0]["mlp"]["shared"].__setitem__("limit", 0.0))
    broken(lambda d: d["layers"][0]["mlp"]["router"].__setitem__("top", 6))
    broken(lambda d: d["layers"][0]["mlp"]["router"].__setitem__("identity", -1))
    broken(lambda d: d["loop"].__setitem__("stop", 4))
    broken(lambda d: d["loop"].__setitem__("stop", 1))
    broken(lambda d: d["loop"].__setitem__("times", 0))
    broken(lambda d: d.pop("norm"))


@pytest.mark.parametrize("loop,want", [
    ((1, 3, 2), [(0, False), (1, True), (2, False), (1, True), (2, False)]),
    ((0, 1, 3), [(0, True), (0, True), (0, True), (1, False), (2, False)]),
    ((0, 3, 2), [(0, True), (1, False), (2, False)] * 2),
    ((2, 3, 1), [(0, False), (1, False), (2, True)]),
    (None, [(0, False), (1, False), (2, False)])])
def test_run_order_joins_and_cache_units(loop, want):
    """The embedding output is joined in front of every pass, the first one too; every layer run has its own unit."""
    import braidinfer_amd as B
    from braidinfer_amd.engine.model import DecoderModel
    d = tiny()
    d.pop("loop")
    if loop is not None:
        d["loop"] = {"start": loop[0], "stop": loop[1], "times": loop[2]}
    cfg = B.config_from_dict(d)
    assert cfg.run_order() == want == P.layer_runs(d)
    model = DecoderModel(B.spec_of(cfg))
    assert [(e.layer, e.input_join is not None) for e in model.schedule] == want
    assert sorted(model.cache_needs()) == list(range(len(want)))
    assert ("loop.in" in {s.name for s in model.weight_specs()}) == (loop is not None)


def test_a_schedule_that_names_no_such_join_is_refused():
    import dataclasses
    import braidinfer_amd as B
    from braidinfer_amd.engine.model import DecoderModel
    from braidinfer_amd.errors import ConfigError
    spec = B.spec_of(B.config_from_dict(tiny()))
    with pytest.raises(ConfigError):
        DecoderModel(dataclasses.replace(spec, input_joins={}))


def test_parts_tensor_names_and_what_the_cache_keeps():
    import braidinfer_amd as B
    from braidinfer_amd.engine.model import DecoderModel
    d = tiny()
    model = DecoderModel(B.spec_of(B.config_from_dict(d)))
    assert {s.name: tuple(s.shape) for s in model.weight_specs()} == P.tensor_shapes(d)
    assert model.graph_safe() and model.state_needs() == {}
    needs = model.cache_needs()
    assert (needs[0].kv_heads, needs[0].key_dim, needs[0].val_dim) == (2, 8, 12)
    assert (needs[1].kv_heads, needs[1].key_dim, needs[1].val_dim) == (1, 18, 14)       # [latent | rotated part], the latent again
    assert needs[1] == needs[3] and needs[2] == needs[4]                                # the two passes of a layer
    # a window of 9: at length 20 the next query (position 20) sees from 12 on; the latent layer sees everything
    assert needs[0].first_live(20) == 12 and needs[1].live_from is None
    assert model.layers[0].mixer.adjacent and model.layers[2].mixer.adjacent
    assert model.layers[1].mixer.halves
    assert model.optional_names() == ["l1.norm2", "l1.ls2", "head.weight"]
    # every key that may be left out
    d2 = copy.deepcopy(d)
    d2.pop("loop")
    for k in ("kv_heads", "vdim", "mask", "rot"):
        d2["layers"][0]["mixer"].pop(k)
    d2["layers"][0]["mlp"].pop("shared")
    d2["layers"][0]["mlp"]["router"].pop("identity")
    d2["layers"][1]["mixer"].update(rot_dim=0)
    d2["layers"][1]["mixer"].pop("rot")
    d2["layers"][1]["mixer"].pop("vdim")
    m2 = DecoderModel(B.spec_of(B.config_from_dict(d2)))
    assert {s.name: tuple(s.shape) for s in m2.weight_specs()} == P.tensor_shapes(d2)
    n2 = m2.cache_needs()
    assert n2[0].live_from is None and (n2[0].kv_heads, n2[0].key_dim, n2[0].val_dim) == (4, 8, 8)
    assert len(m2.positions) == 1


def test_presets_are_configurations():
    import braidinfer_amd as B
    from braidinfer_amd.engine.model import DecoderModel
    for name in ("finosun-tiny", "finosun-1b", "finosun-7b"):
        cfg = B.any_preset(name)
        model = DecoderModel(B.spec_of(cfg))
        assert {s.name: tuple(s.shape) for s in model.weight_specs()} == P.tensor_shapes(cfg.to_dict())


def test_parts_refuse_what_does_not_go_together():
    from braidinfer_amd.config import PartSpec
    from braidinfer_amd.errors import ConfigError
    from braidinfer_amd.parts import build_part
    base = dict(hidden_size=32, intermediate_size=16, num_experts=4, top=2)
    for more in (dict(identity=2), dict(scoring="softmax_all", identity=-1), dict(scoring="softmax_all", limit=0.0), dict(scoring="softmax_all", top=7, identity=2),
                 dict(scoring="softmax_all", shared_size=8, shared_gate=True), dict(scoring="softmax_all", limit=1.0, shared_limit=0.0, shared_size=8)):
        with pytest.raises(ConfigError):
            build_part("feed_forward", PartSpec("routed_experts", dict(base, **more)))
    att = dict(hidden_size=32, num_heads=2, num_kv_heads=1, key_dim=8, value_dim=8, window=4)
    for more in (dict(v_norm_eps=-1.0), dict(v_norm_eps=1e-5, values_from_keys=True), dict(v_norm_eps=1e-5, value_mix="mix")):
        with pytest.raises(ConfigError):
            build_part("mixer", PartSpec("pooled_window_attention", dict(att, **more)))


# ------------------------------------------------------------------ the plain mechanisms against direct sums -------
def test_plain_window():
    T = 23
    for size in (1, 5, 22, 40):
        m = P.window(T, size)
        for i in range(T):
            for j in range(T):
                assert m[i, j] == (0 <= i - j < size)


def test_plain_rotations():
    rng = np.random.default_rng(1)
    x, y = rng.standard_normal((1, 1, 10)), rng.standard_normal((1, 1, 10))
    f = [100 ** (-2 * i / 8) for i in range(4)]
    for neighbours in (True, False):
        a, b = P.turn(x, [7], 8, 100.0, neighbours), P.turn(y, [3], 8, 100.0, neighbours)
        a2, b2 = P.turn(x, [107], 8, 100.0, neighbours), P.turn(y, [103], 8, 100.0, neighbours)
        assert np.allclose(a[..., 8:], x[..., 8:]) and abs(np.linalg.norm(a) - np.linalg.norm(x)) < 1e-12
        assert abs(float((a * b).sum()) - float((a2 * b2).sum())) < 1e-9           # scores depend on distances only
        assert np.allclose(P.turn(x, [0], 8, 100.0, neighbours), x)
        i, j = (2, 3) if neighbours else (1, 5)                                    # pair 1
        u, v, ang = x[0, 0, i], x[0, 0, j], 7 * f[1]
        assert abs(a[0, 0, i] - (u * math.cos(ang) - v * math.sin(ang))) < 1e-12 and abs(a[0, 0, j] - (v * math.cos(ang) + u * math.sin(ang))) < 1e-12


def test_plain_attention_with_a_factor_a_head():
    rng = np.random.default_rng(0)
    T, H, G, d, e = 9, 4, 2, 5, 3
    q, k, v = rng.standard_normal((T, H, d)), rng.standard_normal((T, G, d)), rng.standard_normal((T, G, e))
    scales = 0.7 * np.array([1.0, 0.3, -0.5, 2.0])
    visible = P.window(T, 4)
    got = P.softmax_attention(q, k, v, scales, visible)
    for t in range(T):
        for h in range(H):
            num, den = np.zeros(e), 0.0
            for j in range(max(0, t - 3), t + 1):
                s = math.exp(float(q[t, h] @ k[j, h // 2]) * scales[h])
                num, den = num + s * v[j, h // 2], den + s
            assert np.abs(got[t, h] - num / den).max() < 1e-12


def test_plain_choice_of_outputs_and_clamped_unit():
    rng = np.random.default_rng(2)
    T, N, top = 40, 9, 3
    z, corr = rng.standard_normal((T, N)) * 2, rng.standard_normal(N) * 0.3
    chosen, weights = P.choose_outputs(z, corr, top)
    for t in range(T):
        s = np.exp(z[t]) / np.exp(z[t]).sum()
        want = sorted(range(N), key=lambda e: (-(s[e] + corr[e]), e))[:top]
        assert list(chosen[t]) == want and np.allclose(weights[t], s[want])
    assert weights.sum(axis=1).max() < 1.0                     # not divided by their sum
    h = rng.standard_normal((5, 4))
    gate, up, down = rng.standard_normal((6, 4)) * 2, rng.standard_normal((6, 4)) * 2, rng.standard_normal((3, 6))
    y = P.clamped_unit(h, gate, up, down, 0.9)
    for t in range(5):
        inner = []
        for r in range(6):
            g, u = min(float(gate[r] @ h[t]), 0.9), max(-0.9, min(0.9, float(up[r] @ h[t])))
            inner.append(g / (1 + math.exp(-1.702 * g)) * (u + 1))
        assert np.allclose(y[t], down @ np.array(inner))


def test_plain_latent_mixer_by_absorbed_matrices():
    """The same attention over one row a token: queries through W_uk^T, outputs through W_uv behind the softmax."""
    d = tiny()
    w = P.random_weights(d, 7)
    m, p = d["layers"][1]["mixer"], "l1.mix."
    T, H, dd, r, e, rank = 12, 3, 6, 4, 10, 14
    h = np.random.default_rng(5).standard_normal((T, 40))
    pos = np.arange(T)
    low = h @ w[p + "dkv"].T
    c = P.rms_norm(low[:, :rank], w[p + "dkv.norm"], 1e-4)
    kr = P.turn(low[:, rank:].reshape(T, 1, r), pos, 4, 50.0, False)[:, 0]
    q = (h @ w[p + "q"].T).reshape(T, H, dd + r)
    qr = P.turn(q[..., dd:], pos, 4, 50.0, False)
    uk, uv = w[p + "uk"].reshape(H, dd, rank), w[p + "uv"].reshape(H, e, rank)
    out = np.zeros((T, H, e))
    for i in range(H):
        s = ((q[:, i, :dd] @ uk[i]) @ c.T + qr[:, i] @ kr.T) * m["scale"]
        out[:, i] = (P.softmax(np.where(P.causal(T), s, -np.inf)) @ c) @ uv[i].T
    want = (out.reshape(T, -1) * P.sigmoid(h @ w[p + "g"].T)) @ w[p + "o"].T
    assert np.abs(P.latent_mixer(h, w, p, m, 1e-4, pos) - want).max() < 1e-12


def test_plain_model_is_causal_and_joins_in_front_of_every_pass():
    d = tiny()
    w = P.random_weights(d, 5)
    toks = [int(t) for t in np.random.default_rng(4).integers(0, d["vocab"], 30)]
    whole, rows = P.forward(d, w, toks, return_layers=True)
    assert rows.shape == (5, 30, d["width"])
    assert np.abs(P.forward(d, w, toks[:17]) - whole[:17]).max() < 1e-9
    # a join whose matrix passes the residual rows on is no join; one that takes the embedding output starts a pass over
    w2 = dict(w)
    w2["loop.in"] = np.concatenate([np.eye(40), np.zeros((40, 40))], axis=1)
    once = dict(d, loop={"start": 1, "stop": 3, "times": 1})
    flat = dict(d)
    flat.pop("loop")
    assert np.abs(P.forward(once, w2, toks) - P.forward(flat, w, toks)).max() < 1e-12
    w2["loop.in"] = np.concatenate([np.zeros((40, 40)), np.eye(40)], axis=1)
    assert np.abs(P.forward(d, w2, toks) - P.forward(once, w2, toks)).max() < 1e-12
