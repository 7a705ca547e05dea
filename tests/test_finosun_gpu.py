"""The Finosun design in the engine against the plain implementation (`plain_finosun`): each mechanism's kernels alone,
whole prompts, portions, single tokens, batches, pages and slots used again, keys at the edges of windows and pages and
far away, and greedy generation through the engine's own entry point.  Configurations and weights are made here; where
random weights would hide a fault (one far key among hundreds, an edge that is one token off) they are made so that it
shows."""
import copy
import json
import math
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

import plain_finosun as P

pytestmark = pytest.mark.gpu
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))


def att(heads, kv, dim, vdim=None, size=None, rot=None, scale=None, mlp=None):
    m = {"heads": heads, "kv_heads": kv, "dim": dim, "scale": scale if scale is not None else 1.2 / math.sqrt(dim)}
    if vdim is not None:
        m["vdim"] = vdim
    if size is not None:
        m["mask"] = {"size": size}
    if rot is not None:
        m["rot"] = {"base": rot[1], "dims": rot[0]}
    return {"type": "attention", "mixer": m, "mlp": mlp}


def lat(heads, dim, rot_dim, vdim, rank, base=10000.0, scale=None, mlp=None):
    m = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": rank,
         "scale": scale if scale is not None else 1.0 / math.sqrt(dim + rot_dim)}
    if rot_dim:
        m["rot"] = {"base": base, "dims": rot_dim}
    return {"type": "latent_attention", "mixer": m, "mlp": mlp}


def moe(ff, experts, identity, top, shared=None, limit=1.5, shared_limit=1.0):
    f = {"kind": "moe", "expert": {"ff": ff, "limit": limit}, "router": {"experts": experts, "top": top}}
    if identity is not None:
        f["router"]["identity"] = identity
    if shared is not None:
        f["shared"] = {"ff": shared, "limit": shared_limit}
    return f


def model(width, vocab, layers, loop=None, eps=1e-5):
    d = {"architecture": "Finosun", "vocab": vocab, "width": width, "norm": {"eps": eps}, "layers": layers}
    if loop is not None:
        d["loop"] = {"start": loop[0], "stop": loop[1], "times": loop[2]}
    return d


CONFIGS = {
    # the usual stack: window and latent layers, part of every head rotated, experts with identities and a shared one, a
    # pass in the middle
    "a": model(64, 211, [att(4, 2, 16, 24, 40, (8, 10000.0), mlp=moe(32, 5, 2, 3, 40)), lat(3, 12, 8, 16, 24, mlp=moe(32, 5, 2, 3, 40)),
                         att(6, 2, 16, 16, 70, (12, 500.0), mlp=moe(24, 7, 1, 2, 24, 0.7, 2.0)), lat(2, 16, 16, 24, 40, 300.0, mlp=None)], loop=(1, 3, 2)),
    # sizes the usual shapes make equal or 1, and odd ones: one head, as many kv heads as heads, widths that are no
    # multiples of 4 or 8, a window of one token, no window, no rotation, every element rotated, no rotated key part, a
    # latent wider than the model, all outputs chosen, one chosen, only identities but one expert, no identities, no
    # shared expert, layers without feed-forward, a pass over one layer at the start
    "b": model(50, 97, [lat(1, 5, 2, 7, 9, 40.0, mlp=moe(20, 3, 2, 5, 6)), att(1, 1, 6, 10, 1, (2, 30.0), mlp=moe(10, 1, 5, 2, 13)),
                        att(3, 3, 10, 6, 33, (10, 77.0), mlp=moe(14, 4, None, 1)), lat(3, 6, 0, 5, 61, mlp=moe(9, 2, 1, 1, None, 0.4)),
                        att(5, 1, 7, 9, None, None, mlp=None)], loop=(0, 1, 3), eps=1e-4),
    # sizes that the matrix-core attention kernels, the products' wide tiles and the grouped experts' kernels take; a
    # window that crosses page borders, a pass over the whole model
    "c": model(256, 1000, [att(8, 2, 64, 64, 100, (32, 500000.0), mlp=moe(128, 10, 4, 4, 192, 1.0, 1.5)),
                           lat(4, 64, 32, 64, 96, 500000.0, mlp=moe(128, 10, 4, 4, 192, 1.0, 1.5)),
                           att(4, 4, 128, 96, 65, (48, 10000.0), mlp=moe(128, 10, 4, 4, 192, 1.0, 1.5))], loop=(0, 3, 2)),
    # latent layers only, nothing repeated
    "d": model(64, 101, [lat(2, 16, 8, 16, 32, mlp=moe(16, 3, 1, 2, 16)), lat(4, 8, 4, 12, 20, 100.0, mlp=moe(16, 4, 4, 4))]),
    # attention only, every earlier token seen or a window wider than any prompt here, a scale of 1, one pass at the end
    "e": model(32, 64, [att(2, 2, 16, None, None, (4, 1000.0), scale=1.0, mlp=moe(16, 2, 1, 1)),
                        att(2, 1, 16, 8, 5000, (16, 100.0), scale=1.0, mlp=moe(16, 2, 3, 2, 12))], loop=(1, 2, 1)),
}
GAINS = {"a": 1.0, "b": 1.0, "c": 1.0, "d": 1.0, "e": 0.6}


@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    """(name, dtype) -> (folder, configuration, weights).  The bfloat16 runs get routers whose choice is clear (a token
    that takes another expert than the plain implementation differs by far more than rounding): the corrections lie
    further apart than the scores' whole range; float32 holds the lively ones."""
    out = {}
    for name, cfg in CONFIGS.items():
        for dtype, spread in (("float32", 0.0), ("bfloat16", 2.5)):
            w = P.random_weights(cfg, seed=700 + ord(name), router_spread=spread, gain=GAINS[name])
            d = str(tmp_path_factory.mktemp(f"finosun_{name}_{dtype}"))
            P.write_model(d, cfg, w)
            out[(name, dtype)] = (d, copy.deepcopy(cfg), w)
    return out


@pytest.fixture(scope="module")
def engines(folders):
    import braidinfer_amd as B
    made = {}

    def get(name, dtype, max_tokens=4096):
        if (name, dtype) not in made:
            made[(name, dtype)] = B.Engine.from_folder(folders[(name, dtype)][0], dtype=dtype, max_tokens=max_tokens)
        return made[(name, dtype)]
    return get


_plain = {}


def plain(name, dtype, cfg, w, toks):
    key = (name, dtype, json.dumps(cfg, sort_keys=True), tuple(toks))
    if key not in _plain:
        _plain[key] = P.forward(cfg, w, toks)
    return _plain[key]


def close(got, want, dtype, what=""):
    """Logits against the plain ones: centred difference over the vocabulary, relative to the logits' spread."""
    got, want = np.asarray(got, dtype=np.float64), np.asarray(want)
    assert got.shape == want.shape, f"{what}: {got.shape} against {want.shape}"
    d = got - want
    d = d - d.mean(axis=-1, keepdims=True)
    err = np.sqrt((d * d).mean(axis=-1)) / want.std()
    if dtype == "float32":
        assert err.max() < 1e-4, f"{what}: row {err.argmax()} differs by {err.max():.3g}"
        return
    tol = 6e-2
    assert (err > tol).sum() <= max(1, len(err) // 25) and err.max() < 4 * tol, \
        f"{what}: {int((err > tol).sum())} rows of {len(err)} over {tol}, the worst (row {err.argmax()}) by {err.max():.3g}"


def run(eng, tokens, portions):
    """One sequence in the given portions; logits of every place."""
    import braidinfer_amd as B
    s = eng.alloc_slot()
    out, at = [], 0
    try:
        for n in portions:
            out.append(eng.step([B.StepEntry(s, tokens[at:at + n], list(range(n)))]).cpu().numpy())
            at += n
    finally:
        eng.free_slot(s)
    assert at == len(tokens)
    return np.concatenate(out)


def tokens_of(cfg, n, seed):
    return [int(t) for t in np.random.default_rng(seed).integers(0, cfg["vocab"], n)]


def dev_i(a):
    return torch.tensor(np.asarray(a), dtype=torch.int32).cuda()


def dev_f(a):
    return torch.tensor(np.asarray(a, dtype=np.float32)).cuda()


def dev_16(a):
    return dev_f(a).to(torch.bfloat16)


def host(t):
    return t.float().cpu().numpy().astype(np.float64)


def f32(a):
    """Float64 values that float32 holds exactly."""
    return np.asarray(a, dtype=np.float32).astype(np.float64)


def bf(a):
    return P.to_bf16_values(a)


class Step:
    """What a part alone reads of a step."""

    def __init__(self, n, decode=False):
        from braidinfer_amd.engine.step import Workspace
        self.n_tokens, self.is_decode, self.ws = n, decode, Workspace("cuda")


# ------------------------------------------------------------ mechanisms alone -------
@pytest.mark.parametrize("T,W", [(7, 50), (3, 256), (2, 2050), (2, 4100)])
def test_scaled_rows_that_join_and_the_norm_behind_them(T, W):
    from braidinfer_amd.parts import Runtime, build_part
    from braidinfer_amd.config import PartSpec
    rng = np.random.default_rng(W)
    x, y = rng.standard_normal((T, W)).astype(np.float32), (rng.standard_normal((T, W)) * 3).astype(np.float32)
    s, wn = bf(rng.standard_normal(W)), bf(1 + 0.2 * rng.standard_normal(W))
    want = f32(x) + s * f32(y)
    for dtype, tol in ((torch.float32, 3e-6), (torch.bfloat16, 0.02)):
        rt = Runtime(torch.device("cuda"), dtype)
        part = build_part("norm", PartSpec("layer_scale", {"size": W, "tensor": ""}))
        part.load({"ls": torch.tensor(s, dtype=torch.float32)}, "ls", rt)
        nxt = build_part("norm", PartSpec("rmsnorm", {"size": W, "eps": 1e-3, "tensor": ""}))
        nxt.load({"n": torch.tensor(wn, dtype=torch.float32)}, "n", rt)
        acc = dev_f(x)
        assert not part.add_normed(dev_f(y), acc)
        assert np.abs(host(acc) - want).max() < 3e-6
        acc, out = dev_f(x), torch.zeros((T, W), dtype=dtype, device="cuda")
        assert part.add_normed(dev_f(y), acc, nxt, out)
        assert np.abs(host(acc) - want).max() < 3e-6 and np.abs(host(out) - P.rms_norm(want, wn, 1e-3)).max() < tol
        alone = torch.zeros((T, W), dtype=torch.float32, device="cuda")
        part.forward(dev_f(y), alone)
        assert np.abs(host(alone) - s * f32(y)).max() < 3e-6


@pytest.mark.parametrize("T,W", [(5, 50), (1, 64), (130, 256)])
def test_the_join_with_the_embedding_output(T, W):
    from braidinfer_amd.parts import Runtime, build_part
    from braidinfer_amd.config import PartSpec
    rng = np.random.default_rng(T)
    w_in = bf(rng.standard_normal((W, 2 * W)) / math.sqrt(2 * W))
    x0, x, x_late = bf(rng.standard_normal((T, W))), bf(rng.standard_normal((T, W))), bf(rng.standard_normal((T, W)))
    for dtype, cast in ((torch.float32, dev_f), (torch.bfloat16, dev_16)):
        part = build_part("input_join", PartSpec("linear_join", {"hidden_size": W, "tensor": ""}))
        part.load({"in": cast(w_in)}, "in", Runtime(torch.device("cuda"), dtype))
        step = Step(T)
        part.begin(dev_f(x0), step)
        for rows in (x, x_late):              # several passes of one step read the same embedding output
            acc = dev_f(rows)
            part.forward(acc, step)
            assert np.abs(host(acc) - P.join_input(rows, x0, w_in)).max() < 2e-5


def shuffled_table(n_pages, n_slots, slot, seed):
    """A block table whose pages of `slot` lie in no order among pages that belong to nobody."""
    rng = np.random.default_rng(seed)
    table = np.full((n_slots, n_pages), -1, dtype=np.int32)
    table[slot] = rng.permutation(n_pages + 3)[:n_pages]
    return table


@pytest.mark.parametrize("H,G,d,e,rd", [(4, 2, 16, 24, 8), (3, 3, 10, 6, 10), (1, 1, 6, 20, 0), (8, 2, 64, 64, 32), (4, 4, 128, 96, 48), (2, 1, 130, 200, 2)])
def test_prepare_value_norm_factor_a_head_and_neighbouring_pairs(H, G, d, e, rd):
    """The norm over a token's whole projection, neighbours turned, a factor (of any sign) on a head's queries, every
    head's values over their root mean square, in the query rows and in the cache; in portions that go through the
    kernel of few tokens and the tiled one of many."""
    from braidinfer_amd import kernels as K
    rng = np.random.default_rng(H * 7 + d)
    T, eps = 340, 1e-3
    width = H * d + G * (d + e) + 3
    raw = (rng.standard_normal((T, width)) * 0.05).astype(np.float32)           # small sums: eps inside the root matters
    qn, kn = (1 + 0.3 * rng.standard_normal(H * d)).astype(np.float32), (1 + 0.3 * rng.standard_normal(G * d)).astype(np.float32)
    temps = np.array([1.3, -0.7, 0.0, 2.0, 0.5, 1.0, 3.0, 0.1][:H], dtype=np.float32)
    pos = np.arange(T) + 60                                                      # the pages' border inside
    x = f32(raw)
    q = P.rms_norm(x[:, :H * d], f32(qn), eps).reshape(T, H, d) * f32(temps)[None, :, None]
    k = P.rms_norm(x[:, H * d:(H + G) * d], f32(kn), eps).reshape(T, G, d)
    v = P.rms_divide(x[:, (H + G) * d:(H + G) * d + G * e].reshape(T, G, e), eps)
    freqs = np.array([100.0 ** (-2 * i / rd) for i in range(rd // 2)]) if rd else None
    if rd:
        q, k = P.turn(q, pos, rd, 100.0, True), P.turn(k, pos, rd, 100.0, True)
    n_pages = -(-int(pos[-1] + 1) // 64)
    table = shuffled_table(n_pages, 3, 1, d)
    for dtype, tol in ((torch.float32, 1e-4), (torch.bfloat16, 1e-2)):
        unit = torch.zeros((n_pages + 3, G * 64 * (d + e)), dtype=dtype, device="cuda")
        got_q = []
        for lo, hi in ((0, 41), (41, 42), (42, T)):
            n = hi - lo
            cos = sin = None
            if rd:
                cos, sin = torch.zeros((n, rd // 2), device="cuda"), torch.zeros((n, rd // 2), device="cuda")
                K.rope_table(dev_i(pos[lo:hi]), dev_f(freqs), cos, sin)
            qo = torch.full((n, H * d), 9.0, dtype=dtype, device="cuda")
            K.pwa_prepare(dev_f(raw[lo:hi]), None, dev_f(qn), dev_f(kn), eps, cos, sin, rd, dev_i(pos[lo:hi]), dev_i(np.zeros(n)), dev_i([1]),
                          dev_i(table), qo, unit, None, None, 0, H, G, d, e, 64, True, row_ss=torch.zeros((n, 2), device="cuda"),
                          adjacent=True, q_scale=dev_f(temps), v_eps=eps)
            got_q.append(host(qo))
        assert np.abs(np.concatenate(got_q).reshape(T, H, d) - q).max() < tol * max(1.0, np.abs(q).max())
        pages = host(unit)
        for t in range(T):
            pg = pages[table[1, pos[t] // 64]]
            keys = pg[:G * 64 * d].reshape(G, 64, d)[:, pos[t] % 64]
            vals = pg[G * 64 * d:].reshape(G, e, 64)[:, :, pos[t] % 64]
            assert np.abs(keys - k[t]).max() < tol * max(1.0, np.abs(k).max()), f"keys of token {t}"
            assert np.abs(vals - v[t]).max() < tol * max(1.0, np.abs(v).max()), f"values of token {t}"
        used = set(table[1].tolist())
        assert all(float(np.abs(pages[p]).max()) == 0 for p in range(n_pages + 3) if p not in used)


def test_rotation_in_halves_still_turns_halves():
    from braidinfer_amd import kernels as K
    rng = np.random.default_rng(3)
    T, d, rd = 5, 12, 8
    raw = rng.standard_normal((T, 3 * d)).astype(np.float32)
    table, unit = shuffled_table(1, 1, 0, 0), torch.zeros((4, 64 * 2 * d), device="cuda")
    cos, sin = torch.zeros((T, rd // 2), device="cuda"), torch.zeros((T, rd // 2), device="cuda")
    K.rope_table(dev_i(np.arange(T)), dev_f([50.0 ** (-2 * i / rd) for i in range(rd // 2)]), cos, sin)
    for adjacent in (False, True):
        qo = torch.zeros((T, d), device="cuda")
        K.pwa_prepare(dev_f(raw), None, None, None, 0.0, cos, sin, rd, dev_i(np.arange(T)), dev_i(np.zeros(T)), dev_i([0]), dev_i(table), qo, unit,
                      None, None, 0, 1, 1, d, d, 64, True, adjacent=adjacent)
        assert np.abs(host(qo) - P.turn(f32(raw[:, None, :d]), np.arange(T), rd, 50.0, adjacent)[:, 0]).max() < 1e-5


@pytest.mark.parametrize("H,D,DR,R,T", [(3, 12, 8, 24, 70), (1, 5, 2, 9, 3), (4, 64, 32, 96, 100), (2, 6, 0, 61, 10)])
@pytest.mark.parametrize("halves", [True, False])
def test_latent_rows_and_queries(H, D, DR, R, T, halves):
    """The latent normed, the shared key part and the queries' rotated parts turned, from strided views of one product."""
    from braidinfer_amd import kernels as K
    rng = np.random.default_rng(R)
    eps = 1e-3
    n_q = H * (D + DR)
    raw = (rng.standard_normal((T, n_q + R + DR + 5)) * 0.1).astype(np.float32)
    cw = (1 + 0.3 * rng.standard_normal(R)).astype(np.float32)
    pos = np.arange(T) + 61
    x = f32(raw)
    q, low = x[:, :n_q].reshape(T, H, D + DR), x[:, n_q:n_q + R + DR]
    c, qr, kr = P.rms_norm(low[:, :R], f32(cw), eps), q[..., D:], low[:, R:].reshape(T, 1, DR)
    cos = sin = None
    if DR:
        qr, kr = P.turn(qr, pos, DR, 90.0, not halves), P.turn(kr, pos, DR, 90.0, not halves)
        cos, sin = torch.zeros((T, DR // 2), device="cuda"), torch.zeros((T, DR // 2), device="cuda")
        K.rope_table(dev_i(pos), dev_f([90.0 ** (-2 * i / DR) for i in range(DR // 2)]), cos, sin)
    n_pages = -(-int(pos[-1] + 1) // 64)
    table = shuffled_table(n_pages, 3, 1, R)
    for dtype, tol in ((torch.float32, 3e-5), (torch.bfloat16, 1.5e-2)):
        cache = torch.zeros((n_pages + 3, 64 * (2 * R + DR)), dtype=dtype, device="cuda")
        plain_q, wide_q = torch.zeros((T, H * D), dtype=dtype, device="cuda"), torch.zeros((T, H * (R + DR)), dtype=dtype, device="cuda")
        rows = dev_f(raw)
        K.latent_prepare(rows[:, :n_q], rows[:, n_q:n_q + R + DR], dev_f(cw), eps, cos, sin, DR, dev_i(pos), dev_i(np.zeros(T)), dev_i([1]), dev_i(table),
                         cache, plain_q, wide_q, H, D, DR, R, 64, halves=halves)
        assert np.abs(host(plain_q).reshape(T, H, D) - q[..., :D]).max() < tol
        assert DR == 0 or np.abs(host(wide_q).reshape(T, H, R + DR)[..., R:] - qr).max() < tol
        pages = host(cache)
        for t in range(T):
            pg, row = pages[table[1, pos[t] // 64]], pos[t] % 64
            key = pg[:64 * (R + DR)].reshape(64, R + DR)[row]
            assert np.abs(key[:R] - c[t]).max() < tol * np.abs(c).max() and (DR == 0 or np.abs(key[R:] - kr[t, 0]).max() < tol)
            assert np.array_equal(pg[64 * (R + DR):].reshape(R, 64)[:, row], key[:R])


@pytest.mark.parametrize("T,H,N,Kd", [(1, 3, 16, 24), (70, 4, 64, 96), (5, 2, 7, 9), (33, 1, 200, 40)])
def test_product_head_by_head_with_a_gate(T, H, N, Kd):
    from braidinfer_amd import kernels as K
    rng = np.random.default_rng(N)
    a, w = bf(rng.standard_normal((T, H, Kd))), bf(rng.standard_normal((H, N, Kd)) / math.sqrt(Kd))
    wide = (rng.standard_normal((T, H * N + 5)) * 2).astype(np.float32)
    want = np.einsum("thk,hnk->thn", a, w)
    gated = want * P.sigmoid(f32(wide[:, 5:])).reshape(T, H, N)
    for cast, tol in ((dev_f, 1e-5), (dev_16, 2e-2)):
        out = cast(np.zeros((T, H, N)))
        K.head_linear(cast(a), cast(w), out, gate=dev_f(wide)[:, 5:])
        assert np.abs(host(out) - gated).max() < tol
        K.head_linear(cast(a), cast(w), out)
        assert np.abs(host(out) - want).max() < tol


@pytest.mark.parametrize("T,I", [(5, 24), (3, 7), (130, 64)])
def test_clamped_unit_without_biases_and_with_a_number_a_row(T, I):
    from braidinfer_amd import kernels as K
    rng = np.random.default_rng(I)
    gu = bf(rng.standard_normal((T, 2 * I)) * 2)
    gates = (rng.standard_normal((T, 9)) * 2).astype(np.float32)
    g, u = np.minimum(gu[:, :I], 0.9), np.clip(gu[:, I:], -0.9, 0.9)
    unit = g * P.sigmoid(1.702 * g) * (u + 1)
    assert (gu[:, :I] > 0.9).any() and (gu[:, I:] < -0.9).any()
    for row_gate, want in ((None, unit), (dev_f(gates)[:, 4], unit * P.sigmoid(f32(gates[:, 4:5])))):
        for src, out, tol in ((dev_f(gu), torch.zeros((T, I), device="cuda"), 1e-6), (dev_f(gu), torch.zeros((T, I), dtype=torch.bfloat16, device="cuda"), 8e-3),
                              (dev_16(gu), torch.zeros((T, I), dtype=torch.bfloat16, device="cuda"), 8e-3)):
            K.clamped_glu(src, None, out, 0.9, 1.702, row_gate)
            assert np.abs(host(out) - want).max() < tol


def test_choice_among_all_outputs_by_corrected_softmax_scores():
    from braidinfer_amd import kernels as K
    rng = np.random.default_rng(12)
    for T, N, top in ((40, 12, 4), (30, 64, 8), (9, 5, 5), (9, 6, 1), (20, 70, 5), (11, 130, 8), (3, 512, 64), (1, 3, 2)):
        wide = (rng.standard_normal((T, N + 7)) * 2).astype(np.float32)
        corr = (rng.standard_normal(N) * 0.3 - 0.5).astype(np.float32)          # choice scores below zero happen
        wide[:, 1] = wide[:, 0]
        corr[1] = corr[0]                                                         # two outputs that always tie: the lower number first
        z = f32(wide[:, :N])
        want_c, want_w = P.choose_outputs(z, f32(corr), top)
        chosen = torch.zeros((T, top), dtype=torch.int32, device="cuda")
        share = torch.zeros((T, top), dtype=torch.float32, device="cuda")
        K.route_softmax(dev_f(wide)[:, :N], dev_f(corr), chosen, share, top, 1.0)
        got_c, c = chosen.cpu().numpy(), P.softmax(z) + f32(corr)
        for t in range(T):
            if list(got_c[t]) != list(want_c[t]):
                # float32 scores may order two outputs otherwise than float64 ones only where they are equal to rounding
                assert np.abs(np.sort(c[t][got_c[t]]) - np.sort(c[t][want_c[t]])).max() < 1e-6, f"{N} outputs, token {t}"
            else:
                assert np.abs(share[t].cpu().numpy() - want_w[t]).max() < 1e-6


def experts_part(W, F, E, identity, top, shared, dtype, seed, out_limit=0.8):
    """The feed-forward alone: (part, weights as plain arrays)."""
    from braidinfer_amd.parts import Runtime, build_part
    from braidinfer_amd.config import PartSpec
    rng = np.random.default_rng(seed)
    part = build_part("feed_forward", PartSpec("routed_experts", {
        "hidden_size": W, "intermediate_size": F, "num_experts": E, "top": top, "scoring": "softmax_all", "identity": identity, "limit": out_limit,
        "shared_size": shared, "shared_limit": 1.3 if shared else None, "shared_gate": shared > 0}))
    w = {}
    for s in part.weight_specs("m."):
        w[s.name] = bf(rng.standard_normal(s.shape) * (0.1 if s.name.endswith("correction") else 1.5 / math.sqrt(s.shape[-1])))
    mats = torch.float32 if dtype == torch.float32 else torch.bfloat16
    part.load({n: dev_f(a).to(torch.float32 if n.endswith("correction") else mats) for n, a in w.items()}, "m.", Runtime(torch.device("cuda"), dtype))
    return part, w


def plain_experts(h, w, E, top, shared, limit=0.8):
    f = {"expert": {"limit": limit}, "router": {"experts": E, "top": top}}
    if shared:
        f["shared"] = {"limit": 1.3}
    z = h @ w["m.router"].T
    c = np.sort(P.softmax(z) + w["m.correction"][None, :], axis=1)
    n = c.shape[1]
    clear = np.ones(len(h), dtype=bool) if top == n else c[:, n - top] - c[:, n - top - 1] > 1e-4
    return P.feed_forward(h, w, "m.", f), clear


@pytest.mark.parametrize("W,F,E,identity,top,shared", [(64, 32, 6, 2, 3, 40), (50, 9, 3, 2, 5, 6), (256, 128, 10, 4, 4, 192), (64, 16, 1, 5, 2, 0), (64, 24, 4, 0, 2, 24),
                                                       (128, 64, 70, 10, 6, 64)])
@pytest.mark.parametrize("T,decode", [(1, True), (5, True), (9, False), (60, True), (47, False), (48, False), (300, False)])
def test_experts_identities_and_shared_unit(W, F, E, identity, top, shared, T, decode):
    """Every form of the experts' products (a pair at a time, an expert's weights once, tiles, expert by expert) added to
    rows and stored into them."""
    from braidinfer_amd.parts import ResidualSink
    h = bf(np.random.default_rng(T).standard_normal((T, W)))
    for dtype, cast, tol in ((torch.float32, dev_f, 3e-5), (torch.bfloat16, dev_16, 3e-2)):
        part, w = experts_part(W, F, E, identity, top, shared, dtype, E + F)
        want, clear = plain_experts(h, w, E, top, shared)
        assert clear.mean() > 0.8
        spread = np.sqrt((want ** 2).mean())
        base = np.random.default_rng(3).standard_normal((T, W)).astype(np.float32)
        for forced in ("0", "1"):
            os.environ["BRAIDINFER_EXPERTS_ONE_BY_ONE"] = forced
            try:
                x = dev_f(base)
                part.forward(cast(h), x, Step(T, decode))
                y = torch.full((T, W), 7.0, device="cuda")
                part.forward(cast(h), ResidualSink(y, None, overwrite=True), Step(T, decode))
            finally:
                del os.environ["BRAIDINFER_EXPERTS_ONE_BY_ONE"]
            for got in (host(x) - f32(base), host(y)):
                err = np.abs(got - want).max(axis=1)[clear] / spread
                assert err.max() < tol * 6, f"{dtype}, one by one {forced}: {err.max():.3g}"


@pytest.mark.parametrize("n_pairs", [1, 31, 32, 33, 63, 64, 65, 97, 150])
def test_many_pairs_of_one_expert(n_pairs):
    """An expert's pairs are walked 64 at a time: every count around those borders, beside experts with none and one, and
    pairs of identities behind them."""
    from braidinfer_amd import kernels as K
    rng = np.random.default_rng(n_pairs)
    E, W, F = 4, 136, 72                                 # both inner lengths end inside a run along k
    T = n_pairs + 3
    h = bf(rng.standard_normal((T, W)))
    gu, down = bf(rng.standard_normal((E, 2 * F, W)) / math.sqrt(W)), bf(rng.standard_normal((E, W, F)) / math.sqrt(F))
    ch = np.full((T, 1), 2, dtype=np.int32)
    ch[1], ch[T - 1], ch[0] = 0, E, E + 3                # an expert with one pair, and two identities
    chosen = dev_i(ch)
    first, order, place = dev_i(np.zeros(E + 2)), dev_i(np.zeros(T)), dev_i(np.zeros(T))
    K.experts_sort(chosen, first, order, place, E + 1)
    assert first.tolist() == [0, 1, 1, 1 + n_pairs, 1 + n_pairs, T]
    y = torch.zeros((T, F), dtype=torch.bfloat16, device="cuda")
    K.experts_up_grouped(dev_16(h), dev_16(gu), first, order, y, 1, 0.7, 1.702)
    out = torch.zeros((T, W), device="cuda")
    K.experts_down_grouped(y, dev_16(down), first, out, T)
    x = torch.full((T, W), 3.0, device="cuda")
    share = dev_f(np.linspace(0.5, 1.5, T)[:, None])
    K.experts_combine(out, place, share, x, chosen=chosen, h=dev_16(h), experts=E, store=True)
    want = np.zeros((T, W))
    for t in range(T):
        e = ch[t, 0]
        want[t] = (h[t] if e >= E else P.clamped_unit(h[t:t + 1], gu[e, :F], gu[e, F:], down[e], 0.7)[0]) * float(share[t, 0])
    assert np.abs(host(x) - want).max() < 0.03


def loud_model(kind, size=None):
    """A one-layer model in which token 0's query meets token 1's key with a score far above all others (in the elements
    that are not rotated), and token 1's value moves the logits."""
    W = 48
    layer = att(2, 1, 16, 16, size, (8, 10000.0), scale=1.0) if kind == "attention" else lat(2, 16, 8, 16, 24, scale=1.0)
    cfg = model(W, 60, [layer])
    w = P.random_weights(cfg, 31, gain=0.3)
    w["l0.norm1"], w["l0.ls1"], w["final.norm"] = np.ones(W), np.full(W, 10.0), np.ones(W)      # the mixer outweighs the token itself
    emb = w["embed"] * 0.5
    emb[:, :2] = 0.0
    emb[0, 0] = emb[1, 1] = 12.0                         # element 0 marks the asking token, element 1 the loud one
    w["embed"] = bf(emb)
    big = 3.0 if kind == "attention" else 2.0
    for n in ("q", "k", "dkv"):
        if "l0.mix." + n in w:
            m = w["l0.mix." + n].copy()
            m[:, :2] = 0.0
            w["l0.mix." + n] = m
    if kind == "attention":
        w["l0.mix.q"][12, 0] = w["l0.mix.q"][16 + 12, 0] = big        # element 12 lies behind the rotated ones
        w["l0.mix.k"][12, 1] = big
        w["l0.mix.temp"] = bf(np.array([1.0, 0.8]))
    else:
        w["l0.mix.q"][3, 0] = w["l0.mix.q"][24 + 3, 0] = big
        w["l0.mix.dkv"][5, 1] = big
        uk = w["l0.mix.uk"].copy()
        uk[:, 5] = 0.0
        uk[3, 5] = uk[16 + 3, 5] = 1.5
        w["l0.mix.uk"] = uk
    for n in list(w):
        w[n] = bf(w[n])
    return cfg, w


@pytest.mark.parametrize("kind,size", [("attention", 75), ("attention", 64), ("attention", 65), ("attention", 1), ("attention", 128), ("attention", None),
                                       ("latent", None)])
def test_a_loud_key_at_every_edge(kind, size, tmp_path):
    """One key whose score stands out just inside and just outside the window, at page borders, at the sequence's first
    token and hundreds of tokens away; asked for in a prompt, behind a portion and by a single token."""
    import braidinfer_amd as B
    cfg, w = loud_model(kind, size)
    folder = str(tmp_path / "m")
    P.write_model(folder, cfg, w)
    T = 330
    rng = np.random.default_rng(5)
    cases = []
    for p in (140, 255, 256, 329):
        far = [p - size + 1, p - size, p - size - 1] if size is not None else [0, 1, 63, 64, 127, 128, p - 1]
        cases += [(p, j) for j in far if 0 <= j < p] + ([(p, 0)] if size is not None and p >= size else [])
    for dtype, tol in (("float32", 1e-4), ("bfloat16", 0.05)):
        eng = B.Engine.from_folder(folder, dtype=dtype, max_tokens=1024)
        for p, j in cases:
            toks = [int(t) for t in rng.integers(2, cfg["vocab"], T)]
            toks[p] = 0
            quiet = P.forward(cfg, w, toks[:p + 1])[p]
            toks[j] = 1
            want = P.forward(cfg, w, toks[:p + 1])[p]
            seen = size is None or p - j < size
            moved = np.sqrt(((want - quiet) ** 2).mean()) / quiet.std()
            assert moved > 0.1 if seen else moved < 1e-9, f"the test's key does not show: {moved}"
            for portions in ([p + 1], [p - 1, 2], [p] + [1]):
                got = run(eng, toks[:p + 1], portions)[p]
                err = np.sqrt(((got - want) ** 2).mean()) / want.std()
                assert err < tol, f"{kind} {size} {dtype}: the query at {p} and key {j} ({'seen' if seen else 'unseen'}), portions {portions}: {err:.3g}"
        del eng


# ------------------------------------------------------------ whole models -----------
@pytest.mark.parametrize("name", list(CONFIGS))
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_whole_prompt_against_plain(folders, engines, name, dtype):
    _, cfg, w = folders[(name, dtype)]
    toks = tokens_of(cfg, 150, 1)
    want = plain(name, dtype, cfg, w, toks)
    close(run(engines(name, dtype), toks, [150]), want, dtype, f"{name} {dtype}")
    close(run(engines(name, dtype), toks[:1], [1]), want[:1], dtype, "a sequence of one token")
    close(run(engines(name, dtype), toks[:3], [1, 1, 1]), want[:3], dtype, "the first tokens one by one")
    close(run(engines(name, dtype), toks[:5], [2, 3]), want[:5], dtype, "the first tokens in two portions")


@pytest.mark.parametrize("name", list(CONFIGS))
def test_residual_rows_after_every_layer_run(folders, engines, name):
    import braidinfer_amd as B
    _, cfg, w = folders[(name, "float32")]
    toks = tokens_of(cfg, 60, 9)
    _, layers = P.forward(cfg, w, toks, return_layers=True)
    eng = engines(name, "float32")
    seen = {}
    s = eng.alloc_slot()
    eng.step([B.StepEntry(s, toks, [])], probe=lambda n, t: seen.__setitem__(n, t.float().cpu().numpy().copy()))
    eng.free_slot(s)
    assert len(layers) == len(P.layer_runs(cfg))
    for i in range(len(layers)):
        assert np.abs(seen[f"L{i}.post_ffn"] - layers[i]).max() < 1e-4 * np.abs(layers[i]).max(), f"layer run {i}"


@pytest.mark.parametrize("name", list(CONFIGS))
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_portions_and_single_tokens(folders, engines, name, dtype):
    """A prompt in portions down to two tokens, then token by token across pages' borders and windows' edges, against the
    plain logits and, in float32, against the whole prompt's own."""
    _, cfg, w = folders[(name, dtype)]
    n = 215
    toks = tokens_of(cfg, n, 2)
    want = plain(name, dtype, cfg, w, toks)
    eng = engines(name, dtype)
    whole = run(eng, toks, [n])
    for portions in ([2, 3, 59, 1, 63, 2, 64, 21], [17] + [1] * 198, [128, 2] + [1] * 85):
        got = run(eng, toks, portions)
        close(got, want, dtype, f"{name} {dtype} {portions[:4]}")
        if dtype == "float32":
            assert np.abs(got - whole).max() < 1e-4 * np.abs(whole).max()


@pytest.mark.parametrize("name", ["a", "b", "c"])
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_unequal_batch_against_each_alone(folders, engines, name, dtype):
    import braidinfer_amd as B
    _, cfg, w = folders[(name, dtype)]
    eng = engines(name, dtype)
    lens = [1, 90, 33, 140, 7]
    prompts = [tokens_of(cfg, n + 20, 10 + n) for n in lens]
    slots = [eng.alloc_slot() for _ in lens]
    got = [[] for _ in lens]
    lg = eng.step([B.StepEntry(s, p[:n], list(range(n))) for s, p, n in zip(slots, prompts, lens)]).cpu().numpy()
    at = 0
    for i, n in enumerate(lens):
        got[i].append(lg[at:at + n])
        at += n
    live = list(range(len(lens)))
    for t in range(20):
        if t == 8:                                  # two requests end early; the batch goes on without them
            for i in (1, 4):
                eng.free_slot(slots[i])
                live.remove(i)
        lg = eng.step([B.StepEntry(slots[i], [prompts[i][lens[i] + t]], [0]) for i in live]).cpu().numpy()
        for r, i in enumerate(live):
            got[i].append(lg[r:r + 1])
    for i in live:
        eng.free_slot(slots[i])
    for i, p in enumerate(prompts):
        g = np.concatenate(got[i])
        close(g, plain(name, dtype, cfg, w, p)[:len(g)], dtype, f"request {i} of the batch")


def test_mixed_steps_of_prompts_portions_and_single_tokens(folders, engines):
    """A step may bring a whole prompt, a portion and single tokens at once (the engine's own scheduler does)."""
    import braidinfer_amd as B
    for dtype in ("float32", "bfloat16"):
        _, cfg, w = folders[("a", dtype)]
        eng = engines("a", dtype)
        seqs = [tokens_of(cfg, 100, 200 + i) for i in range(3)]
        s = [eng.alloc_slot() for _ in seqs]
        eng.step([B.StepEntry(s[0], seqs[0][:63], []), B.StepEntry(s[1], seqs[1][:2], [])])
        lg = eng.step([B.StepEntry(s[0], [seqs[0][63]], [0]), B.StepEntry(s[1], seqs[1][2:70], [0, 67]), B.StepEntry(s[2], seqs[2][:41], [40])]).cpu().numpy()
        lg2 = eng.step([B.StepEntry(s[2], seqs[2][41:43], [1]), B.StepEntry(s[0], [seqs[0][64]], [0])]).cpu().numpy()
        for i in s:
            eng.free_slot(i)
        r = [P.forward(cfg, w, q) for q in seqs]
        close(np.concatenate([lg, lg2]), np.stack([r[0][63], r[1][2], r[1][69], r[2][40], r[2][42], r[0][64]]), dtype, f"mixed steps {dtype}")


def test_slots_and_pages_used_again(folders):
    """Requests come and go through a cache of few pages and slots: what a returned page held never shows, the window's
    pages go back while the latent layers' stay, and every page comes back."""
    import braidinfer_amd as B
    folder, cfg, w = folders[("a", "float32")]
    eng = B.Engine.from_folder(folder, dtype="float32", max_tokens=448, max_seq_len=448, n_slots=2)
    free_before = [g.pool.free_count for g in eng.cache.groups]
    assert sorted(eng.cache.group_of_unit) == list(range(6))           # one unit a layer run
    for r in range(5):
        toks = tokens_of(cfg, 120 + 67 * r, 50 + r)
        close(run(eng, toks, [len(toks) - 10] + [1] * 10), P.forward(cfg, w, toks), "float32", f"request {r}")
    assert [g.pool.free_count for g in eng.cache.groups] == free_before
    toks = tokens_of(cfg, 400, 77)
    s = eng.alloc_slot()
    got = [eng.step([B.StepEntry(s, toks[:380], [379])]).cpu().numpy()]
    held = lambda u: [i for i, p in enumerate(eng.cache.unit_group(u).pages[s]) if p >= 0]
    assert held(0) == [5] and held(1) == held(3) == list(range(6)) and held(2) == held(4) == [4, 5]
    for t in range(380, 400):
        got.append(eng.step([B.StepEntry(s, [toks[t]], [0])]).cpu().numpy())
    eng.free_slot(s)
    close(np.concatenate(got), P.forward(cfg, w, toks)[379:], "float32", "behind returned pages")
    # two requests side by side whose slots have just been used, one of them a single token long
    a, b = tokens_of(cfg, 70, 90), tokens_of(cfg, 1, 91)
    sa, sb = eng.alloc_slot(), eng.alloc_slot()
    lg = eng.step([B.StepEntry(sa, a, [69]), B.StepEntry(sb, b, [0])]).cpu().numpy()
    eng.free_slot(sa)
    eng.free_slot(sb)
    close(lg, np.stack([P.forward(cfg, w, a)[69], P.forward(cfg, w, b)[0]]), "float32", "after the slots' earlier users")


@pytest.mark.parametrize("name", ["a", "b", "c"])
def test_long_decoding(folders, engines, name):
    """Three hundred single-token steps from a short prompt (recorded steps of the engine), past page borders, with
    windows that move over decoded tokens."""
    for dtype in ("float32", "bfloat16"):
        _, cfg, w = folders[(name, dtype)]
        toks = tokens_of(cfg, 330, 3)
        close(run(engines(name, dtype), toks, [30] + [1] * 300), plain(name, dtype, cfg, w, toks), dtype, f"{name} {dtype}")


def test_a_long_prompt(folders, engines):
    for dtype in ("float32", "bfloat16"):
        _, cfg, w = folders[("c", dtype)]
        toks = tokens_of(cfg, 700, 8)
        want = plain("c", dtype, cfg, w, toks)
        close(run(engines("c", dtype), toks, [700]), want, dtype, f"whole {dtype}")
        close(run(engines("c", dtype), toks, [100, 600]), want, dtype, f"behind a portion {dtype}")


def drawn_configuration(seed):
    """A configuration drawn at random: any order of layers and passes, head counts and widths from lists that hold odd
    ones and such that the matrix-core kernels take, any window, keys left out."""
    rng = np.random.default_rng(seed)
    pick = lambda xs: xs[int(rng.integers(len(xs)))]

    def mlp():
        if rng.random() < 0.15:
            return None
        E, ident = pick([1, 2, 4, 6, 16]), pick([None, 1, 2, 5])
        top = pick([t for t in (1, 2, 3, 4, 8) if t <= E + (ident or 0)])
        return moe(pick([8, 16, 20, 40]), E, ident, top, pick([None, 16, 24]), pick([0.5, 1.0, 7.0]), pick([0.5, 2.0]))
    layers = []
    for _ in range(int(rng.integers(2, 6))):
        if rng.random() < 0.5:
            H = pick([1, 2, 3, 4, 6, 8, 12])
            G = pick([g for g in (1, 2, 3, 4, 6, 8, 12) if H % g == 0])
            d = pick([8, 12, 16, 24, 32, 64])
            rot = (pick([r for r in (2, 4, 8, 12, 16, 32, 64) if r <= d]), pick([100.0, 10000.0, 1e6])) if rng.random() < 0.85 else None
            layers.append(att(H, G, d, pick([None, 8, 12, 16, 32, 64]), pick([None, 1, 7, 33, 64, 100]), rot, mlp=mlp()))
        else:
            layers.append(lat(pick([1, 2, 3, 4, 8, 12]), pick([4, 8, 12, 16, 32, 64]), pick([0, 2, 4, 8, 16, 32]), pick([4, 8, 12, 32, 64]),
                              pick([7, 16, 24, 64, 128, 200]), pick([100.0, 10000.0]), mlp=mlp()))
    n = len(layers)
    a = int(rng.integers(0, n))
    loop = (a, int(rng.integers(a + 1, n + 1)), pick([1, 2, 3])) if rng.random() < 0.75 else None
    return model(pick([32, 48, 50, 64, 80]), int(rng.integers(40, 300)), layers, loop, eps=pick([1e-6, 1e-5, 1e-3]))


@pytest.mark.parametrize("seed", range(14))
def test_configurations_drawn_at_random(seed, tmp_path):
    """Whole, in portions and token by token in float32 against the plain implementation; bfloat16 whole and decoded."""
    import braidinfer_amd as B
    cfg = drawn_configuration(3000 + seed)
    what = f"seed {seed}: {json.dumps(cfg)}"
    toks = tokens_of(cfg, 110, seed)
    other = tokens_of(cfg, 45, seed + 50)
    folder = str(tmp_path / "m")
    w = P.random_weights(cfg, seed=seed, gain=0.9)
    P.write_model(folder, cfg, w)
    want, ow = P.forward(cfg, w, toks), P.forward(cfg, w, other)
    eng = B.Engine.from_folder(folder, dtype="float32", max_tokens=512)
    close(run(eng, toks, [110]), want, "float32", what)
    close(run(eng, toks, [3, 62, 2, 1, 1] + [1] * 41), want, "float32", what + " in portions")
    sa, sb = eng.alloc_slot(), eng.alloc_slot()
    lg = eng.step([B.StepEntry(sa, toks[:70], [69]), B.StepEntry(sb, other[:44], [0, 43])]).cpu().numpy()
    lg2 = eng.step([B.StepEntry(sa, toks[70:71], [0]), B.StepEntry(sb, other[44:], [0])]).cpu().numpy()
    eng.free_slot(sa)
    eng.free_slot(sb)
    close(np.concatenate([lg, lg2]), np.stack([want[69], ow[0], ow[43], want[70], ow[44]]), "float32", what + " two requests")
    del eng
    w = P.random_weights(cfg, seed=seed, gain=0.9, router_spread=2.5)
    P.write_model(folder, cfg, w)
    eng = B.Engine.from_folder(folder, dtype="bfloat16", max_tokens=512)
    close(run(eng, toks, [60] + [1] * 50), P.forward(cfg, w, toks), "bfloat16", what + " bfloat16")


def test_greedy_generation_through_the_engine(folders, engines):
    _, cfg, w = folders[("a", "float32")]
    prompts = [tokens_of(cfg, n, 20 + n) for n in (3, 41, 12, 70)]
    want = [P.greedy(cfg, w, p, 12) for p in prompts]
    got = engines("a", "float32").generate(prompts, max_new_tokens=12, temperature=0.0, stop_token_ids=[])
    assert got == want
    _, cfg, w = folders[("a", "bfloat16")]
    want = [P.greedy(cfg, w, p, 12) for p in prompts]
    got16 = engines("a", "bfloat16").generate(prompts, max_new_tokens=12, temperature=0.0, stop_token_ids=[])
    for g, wnt, p in zip(got16, want, prompts):
        for i, (a, b) in enumerate(zip(g, wnt)):
            if a != b:                              # bfloat16 may take the runner-up where two logits are nearly tied
                l = P.forward(cfg, w, p + wnt[:i])[-1]
                assert abs(l[a] - l[b]) < 0.05 * np.abs(l).max()
                break


def test_the_command_line_generates_from_a_finosun_folder(folders):
    """`bin/generate` on a Finosun folder: the model class by config.json, greedy tokens as the plain implementation's; a
    sampled run ends and stays inside the vocabulary."""
    folder, cfg, w = folders[("a", "float32")]
    p = [7, 3, 200, 5, 11]
    want = P.greedy(cfg, w, p, 6)
    env = dict(os.environ, MODEL=folder, MAX_TOKENS="6")
    gen = [sys.executable, os.path.join(ROOT, "bin", "generate"), "--dtype", "float32", "--prompt-ids", ",".join(map(str, p))]
    r = subprocess.run(gen, env=env, capture_output=True, text=True)
    assert r.returncode == 0, r.stderr
    assert [int(t) for t in r.stdout.split()] == want
    r = subprocess.run(gen + ["--temperature", "0.8", "--top-k", "20", "--seed", "5"], env=env, capture_output=True, text=True)
    assert r.returncode == 0, r.stderr
    toks = [int(t) for t in r.stdout.split()]
    assert len(toks) == 6 and all(0 <= t < cfg["vocab"] for t in toks)


def test_presets_run(tmp_path):
    """The tiny preset as a random-weights folder of the library's own making, against the plain implementation."""
    import braidinfer_amd as B
    cfg = B.any_preset("finosun-tiny")
    folder = B.Engine.write_random_folder(str(tmp_path / "m"), cfg, seed=3, std=0.1, vector_jitter=0.3)
    pc, pw = P.read_model(folder)
    toks = tokens_of(pc, 120, 4)
    eng = B.Engine.from_folder(folder, dtype="float32", max_tokens=512)
    close(run(eng, toks, [90] + [1] * 30), P.forward(pc, pw, toks), "float32", "preset")


def test_replay_of_given_tokens_through_the_command(folders, tmp_path):
    """`bin/trace_run` as a child process on a Finosun folder: requests whole, with their last tokens one by one, and two
    of unequal length in one batch, against the plain logits."""
    folder, cfg, w = folders[("b", "float32")]
    V = cfg["vocab"]
    seqs = [tokens_of(cfg, n, 60 + n) for n in (90, 41)]
    refs = [P.forward(cfg, w, s) for s in seqs]
    out = str(tmp_path / "out")
    p = subprocess.Popen([sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model", folder, "--dtype", "float32", "--out", out,
                          "--max-tokens", "512"], stdin=subprocess.PIPE, stdout=subprocess.PIPE, text=True)
    n = [0]

    def step(entries, end=()):
        p.stdin.write(json.dumps({"step": n[0], "entries": entries, "end": list(end)}) + "\n")
        p.stdin.flush()
        line = p.stdout.readline().strip()
        assert line == f"done {n[0]}", f"trace_run said {line!r} (exit {p.poll()})"
        path = os.path.join(out, f"{n[0]}.f32")
        n[0] += 1
        return np.fromfile(path, dtype="<f4").reshape(-1, V) if os.path.exists(path) else None

    got = step([{"id": "w", "tokens": seqs[0], "want": [0, 63, 64, 89]}], end=["w"])
    close(got, refs[0][[0, 63, 64, 89]], "float32", "whole")
    assert step([{"id": "d", "tokens": seqs[0][:60], "want": []}]) is None
    for t in range(60, 90):
        got = step([{"id": "d", "tokens": [seqs[0][t]], "want": [0]}], end=["d"] if t == 89 else [])
        close(got, refs[0][t:t + 1], "float32", f"one by one at {t}")
    got = step([{"id": "a", "tokens": seqs[0][:80], "want": [79]}, {"id": "b", "tokens": seqs[1][:35], "want": [3, 34]}])
    close(got, np.stack([refs[0][79], refs[1][3], refs[1][34]]), "float32", "a batch's prompts")
    for t in range(6):
        ending = ["b"] if t == 5 else []
        got = step([{"id": "a", "tokens": [seqs[0][80 + t]], "want": [0]}, {"id": "b", "tokens": [seqs[1][35 + t]], "want": [0]}], end=ending)
        close(got, np.stack([refs[0][80 + t], refs[1][35 + t]]), "float32", f"a batch's token {t}")
    p.stdin.close()
    assert p.wait(timeout=60) == 0
