"""The Tuzisun design in the engine against the plain implementation (`plain_tuzisun`): each mechanism's kernels alone,
whole prompts, portions, single tokens, batches, pages and slots used again, keys at the edges of windows and pages, a
token remembered from far away, and greedy generation through the engine's own entry point.  Configurations and weights
are made here; where random weights would hide a fault (one far key among hundreds, an edge that is one token off) they
are made so that it shows."""
import copy
import json
import math
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

import plain_tuzisun as P

pytestmark = pytest.mark.gpu
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))


def par(heads, kv, dim, vdim, size, rot, ssm, scales=(0.7, 1.2), mlp=None, scale=None):
    """A parallel layer; `ssm` = (heads, vdim, state, groups, norm_groups, taps)."""
    left = {"heads": heads, "kv_heads": kv, "dim": dim, "scale": scale if scale is not None else 1.2 / math.sqrt(dim)}
    if vdim is not None:
        left["vdim"] = vdim
    if size is not None:
        left["mask"] = {"size": size}
    if rot is not None:
        left["rot"] = {"base": rot[1], "dims": rot[0]}
    right = dict(zip(("heads", "vdim", "state", "groups", "norm_groups", "conv"), ssm))
    return {"type": "parallel", "mixer": {"left": left, "left_scale": scales[0], "right": right, "right_scale": scales[1]}, "mlp": mlp}


def mls(heads, dim, vdim, cap=6.0, mlp=None):
    return {"type": "mlstm", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "gate_cap": cap}, "mlp": mlp}


def cdr(heads, kv, dim, vdim, taps, mlp=None):
    return {"type": "channel_delta", "mixer": {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "conv": taps}, "mlp": mlp}


def dense(ff, limit=1.5):
    return {"kind": "dense", "ff": ff, "limit": limit}


def moe(ff, experts, top, groups=None):
    r = {"experts": experts, "top": top}
    if groups is not None:
        r["groups"] = {"count": groups[0], "keep": groups[1]}
    return {"kind": "moe", "expert": {"ff": ff}, "router": r}


def model(width, vocab, streams, layers, eps=1e-5):
    return {"architecture": "Tuzisun", "vocab": vocab, "width": width, "streams": streams, "norm": {"eps": eps}, "layers": layers}


CONFIGS = {
    # the usual stack in another order: every mixer, clamped units and experts, part of every head rotated
    "a": model(72, 211, 3, [mls(3, 16, 24, mlp=moe(32, 6, 2, (3, 2))), par(4, 2, 16, 24, 40, (8, 10000.0), (4, 12, 20, 2, 2, 4), mlp=dense(56)),
                            cdr(4, 2, 16, 24, 4, mlp=moe(24, 8, 3, (2, 1))), par(6, 3, 16, 16, 70, (12, 500.0), (6, 16, 16, 3, 4, 3), mlp=None)]),
    # sizes the usual shapes make equal or 1, and odd ones: one stream, one head, as many kv heads as heads, widths that are no
    # multiples of 4 or 8, a window of one token, no window, no rotation, every element rotated, one tap, all experts chosen,
    # one chosen, groups of one expert, no groups, layers without feed-forward
    "b": model(50, 97, 1, [par(1, 1, 6, 10, 1, (2, 30.0), (1, 5, 7, 1, 1, 1), (1.0, 1.0), mlp=moe(10, 5, 5)), cdr(1, 1, 5, 9, 1, mlp=dense(21, 0.5)),
                           par(3, 3, 10, 6, None, None, (3, 7, 3, 3, 7, 2), (-0.6, 0.9), mlp=None), mls(1, 7, 1, 2.0, mlp=moe(14, 4, 1, (4, 3))),
                           cdr(3, 3, 6, 6, 5, mlp=None), mls(2, 1, 5, 20.0, mlp=moe(9, 3, 2)), par(5, 1, 7, 7, 33, (6, 77.0), (2, 9, 17, 1, 2, 6), mlp=dense(30, 3.0))],
               eps=1e-4),
    # sizes that the matrix-core attention kernels, the products' wide tiles and the grouped experts' kernels take; a window
    # that crosses page borders
    "c": model(512, 1000, 2, [par(8, 2, 64, 64, 100, (32, 500000.0), (8, 64, 64, 2, 4, 4), mlp=dense(384)), mls(4, 64, 128, 15.0, mlp=moe(128, 12, 4, (4, 2))),
                              cdr(8, 4, 64, 64, 4, mlp=moe(128, 12, 4, (4, 3))), par(4, 4, 128, 96, 65, (128, 10000.0), (4, 128, 128, 1, 1, 4), mlp=dense(320))]),
    # recurrent layers only, five streams
    "d": model(64, 101, 5, [cdr(6, 3, 8, 12, 3, mlp=moe(16, 4, 2, (2, 2))), mls(4, 8, 8, 10.0, mlp=dense(40)), cdr(2, 1, 24, 16, 2, mlp=None)]),
    # parallel layers only, more heads than a wave has lanes, wide states
    "e": model(48, 64, 2, [par(2, 1, 16, 8, 5000, (16, 100.0), (66, 2, 130, 11, 3, 4), scale=0.8, mlp=dense(24)),
                           par(12, 4, 8, 8, 64, (4, 1000.0), (4, 3, 300, 2, 1, 2), scale=0.8, mlp=moe(16, 9, 3, (3, 3)))]),
}
GAINS = {"a": 1.0, "b": 1.0, "c": 1.0, "d": 1.0, "e": 0.8}
RANKS = {"a": (5, 7), "b": (1, 3), "c": (32, 24), "d": (9, 4), "e": (5, 7)}


@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    """(name, dtype) -> (folder, configuration, weights).  The bfloat16 runs get routers whose choice is clear (a token
    that takes another expert than the plain implementation differs by far more than rounding), and no matrix memory whose
    heads have one channel (divided by its own root mean square it is a sign); float32 holds the lively ones."""
    out = {}
    for name, given in CONFIGS.items():
        for dtype, spread in (("float32", None), ("bfloat16", 0.5)):
            cfg = copy.deepcopy(given)
            for l in cfg["layers"] if dtype == "bfloat16" else []:
                if l["type"] == "mlstm":
                    l["mixer"].update(dim=max(6, l["mixer"]["dim"]), vdim=max(6, l["mixer"]["vdim"]))
            w = P.random_weights(cfg, seed=900 + ord(name), router_spread=spread, gain=GAINS[name], ranks=RANKS[name])
            d = str(tmp_path_factory.mktemp(f"tuzisun_{name}_{dtype}"))
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


def row_errors(got, want):
    """Centred difference over the vocabulary per row, relative to the logits' spread."""
    d = np.asarray(got, dtype=np.float64) - want
    d = d - d.mean(axis=-1, keepdims=True)
    return np.sqrt((d * d).mean(axis=-1)) / want.std()


_rounded = {}


def rounded(cfg, w, toks, dtype):
    """How far rounding the halves' inputs alone moves the plain logits, per row (None in float32): heads of one or three
    channels that are divided by their own root mean square turn a rounding into another sign."""
    if dtype == "float32":
        return None
    key = (json.dumps(cfg, sort_keys=True), tuple(toks))
    if key not in _rounded:
        _rounded[key] = row_errors(P.forward(cfg, w, toks, round_inputs=True), P.forward(cfg, w, toks))
    return _rounded[key]


def close(got, want, dtype, what="", moved=None):
    """Logits against the plain ones, row by row.  `moved`: what `rounded` says of these rows."""
    want = np.asarray(want)
    assert np.asarray(got).shape == want.shape, f"{what}: {np.asarray(got).shape} against {want.shape}"
    err = row_errors(got, want)
    if dtype == "float32":
        assert err.max() < 1e-4, f"{what}: row {err.argmax()} differs by {err.max():.3g}"
        return
    tol = 6e-2
    over, most = len(err) // 25, 4 * tol
    if moved is not None:
        over, most = max(over, 4 * int((moved > tol).sum())), max(most, 4 * moved.max())
    assert (err > tol).sum() <= max(1, over) and err.max() < most, \
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


def from_slot(t, slot):
    return host(t[slot])


# ------------------------------------------------------------ mechanisms alone -------
@pytest.mark.parametrize("S", [1, 2, 3, 4, 5, 9, 16])
@pytest.mark.parametrize("T,W", [(7, 50), (3, 256), (1, 64), (40, 132)])
def test_streams_spread_open_and_join(S, T, W):
    """Weighted sums, mixing [from, to], one and two branches with biases and scales, the norm behind them, chosen rows."""
    from braidinfer_amd import kernels as K
    rng = np.random.default_rng(100 * S + W)
    x = f32(rng.standard_normal((T, W)))
    X0 = torch.zeros((T, S * W), device="cuda")
    K.streams_spread(dev_f(x), X0, S)
    assert np.array_equal(host(X0).reshape(T, S, W), np.repeat(x[:, None], S, axis=1))
    X = f32(rng.standard_normal((T, S, W)))
    cin, cout, mix, nin = (f32(rng.standard_normal(n)) for n in ((S,), (S,), (S, S), (S,)))
    w = {"n": f32(1 + 0.2 * rng.standard_normal(W)), "n.b": f32(0.3 * rng.standard_normal(W)), "n.alpha": f32(0.7)}
    norm = (dev_f([w["n.alpha"]]), dev_f(w["n"]), dev_f(w["n.b"]))
    coef = dev_f(np.concatenate([cin, cout, mix.reshape(-1)]))
    y1, y2, b1, b2 = (f32(rng.standard_normal(n)) for n in ((T, W), (T, W), (W,), (W,)))
    for branches, y in (([(y1, None, 1.0)], y1), ([(y1, b1, 0.6)], 0.6 * (y1 + b1)), ([(y1, b1, -0.5), (y2, None, 1.5)], -0.5 * (y1 + b1) + 1.5 * y2),
                        ([(y1, None, 0.3), (y2, b2, 1.0)], 0.3 * y1 + y2 + b2)):
        new = np.einsum("tsw,sr->trw", X, mix) + cout[None, :, None] * y[:, None]
        u = np.einsum("trw,r->tw", new, nin)
        dev = [(dev_f(r), None if b is None else dev_f(b), s) for r, b, s in branches]
        for dtype, tol in ((torch.float32, 3e-5), (torch.bfloat16, 0.02)):
            for with_norm in (True, False):
                got, h = dev_f(X.reshape(T, S * W)), torch.zeros((T, W), dtype=dtype, device="cuda")
                K.streams_join(got, coef, dev, S, h, dev_f(nin), norm if with_norm else None)
                assert np.abs(host(got).reshape(T, S, W) - new).max() < 3e-5
                want = P.dynamic_tanh(u, w, "n") if with_norm else u
                assert np.abs(host(h) - want).max() < tol * max(1.0, np.abs(want).max())
        alone = dev_f(X.reshape(T, S * W))
        K.streams_join(alone, coef, dev, S)
        assert np.abs(host(alone).reshape(T, S, W) - new).max() < 3e-5
    rows = [T - 1, 0, T // 2]
    for dtype, tol in ((torch.float32, 2e-5), (torch.bfloat16, 0.02)):
        h = torch.zeros((T, W), dtype=dtype, device="cuda")
        K.streams_open(dev_f(X.reshape(T, S * W)), h, S, coef, norm)
        want = P.dynamic_tanh(np.einsum("tsw,s->tw", X, cin), w, "n")
        assert np.abs(host(h) - want).max() < tol * max(1.0, np.abs(want).max())
        h = torch.zeros((3, W), dtype=dtype, device="cuda")
        K.streams_open(dev_f(X.reshape(T, S * W)), h, S, rows=dev_i(rows))
        assert np.abs(host(h) - X.sum(axis=1)[rows]).max() < tol * 8


def test_tanh_norm_as_a_part():
    from braidinfer_amd.config import PartSpec
    from braidinfer_amd.parts import Runtime, build_part
    rng = np.random.default_rng(0)
    W = 70
    w = {"n": bf(rng.standard_normal(W)), "n.b": bf(rng.standard_normal(W)), "n.alpha": bf(1.3)}
    part = build_part("norm", PartSpec("dynamic_tanh", {"size": W, "tensor": ""}))
    assert {s.name for s in part.weight_specs("n")} == set(w)
    part.load({n: torch.tensor(a, dtype=torch.float32) for n, a in w.items()}, "n", Runtime(torch.device("cuda"), torch.float32))
    x = f32(rng.standard_normal((5, W)) * 2)
    out = torch.zeros((5, W), device="cuda")
    assert np.abs(host(part.forward(dev_f(x), out)) - P.dynamic_tanh(x, w, "n")).max() < 2e-6
    two = torch.zeros((2, W), device="cuda")
    assert np.abs(host(part.forward(dev_f(x), two, rows=dev_i([3, 1]))) - P.dynamic_tanh(x, w, "n")[[3, 1]]).max() < 2e-6


def batch(lengths, slots):
    """(sequence of token, offsets, slots) of packed sequences."""
    return dev_i(np.repeat(np.arange(len(lengths)), lengths)), dev_i(np.concatenate([[0], np.cumsum(lengths)])), dev_i(slots)


@pytest.mark.parametrize("C,H,n,strided", [(20, 3, 4, 0), (7, 2, 3, 1), (64, 5, 1, 4), (132, 66, 6, 8), (12, 1, 16, 0), (9, 4, 2, 3)])
def test_state_space_inputs_in_portions(C, H, n, strided):
    """The convolution with its kept inputs in slots that are not neighbours, beside a padding sequence, in portions of
    many, two and one token (whose kept inputs the kernel itself brings up to date), and the decay and step size."""
    from braidinfer_amd import kernels as K
    rng = np.random.default_rng(C + n)
    lens = [23, 9]
    width = C + H + strided
    taps, bias = f32(rng.standard_normal((C, n))), f32(rng.standard_normal(C))
    a_log, dt_bias = f32(rng.standard_normal(H)), f32(rng.standard_normal(H))
    raw = [f32(rng.standard_normal((L, width)) * (1 if i else 2)) for i, L in enumerate(lens)]
    raw[0][3, C] = 30.0                                         # softplus where it is the identity
    want = [P.short_convolution(r[:, :C], taps, bias) for r in raw]
    kept = torch.zeros((5, max(1, (n - 1) * C) + 3), device="cuda")
    state = kept[:, 3:3 + (n - 1) * C] if n > 1 else None
    at = [0, 0]
    for take in ([5, 1], [1, 1], [1, 2], [2, 1], [1, 1], [13, 3]):
        pad = np.zeros((1, width))
        rows = dev_f(np.concatenate([raw[0][at[0]:at[0] + take[0]], pad, raw[1][at[1]:at[1] + take[1]]]))
        sot, cu, slots = batch([take[0], 1, take[1]], [3, -1, 1])
        T = sum(take) + 1
        out, gb = torch.full((T, C), 9.0, device="cuda"), torch.full((T, 2 * H), 9.0, device="cuda")
        K.ssm_prepare(rows[:, :C], dev_f(taps.T.copy()), dev_f(bias), state, rows[:, C:C + H], dev_f(a_log), dev_f(dt_bias), sot, cu, slots, out, gb, 3,
                      single_tokens=max(take) == 1)
        got, g = host(out), host(gb)
        for i, lo in ((0, 0), (1, take[0] + 1)):
            assert np.abs(got[lo:lo + take[i]] - want[i][at[i]:at[i] + take[i]]).max() < 1e-5, f"sequence {i} at {at[i]}"
            s = P.softplus(raw[i][at[i]:at[i] + take[i], C:C + H] + dt_bias)
            assert np.abs(g[lo:lo + take[i], H:] - s).max() < 1e-5 and np.abs(g[lo:lo + take[i], :H] - np.exp(-np.exp(a_log) * s)).max() < 1e-5
            at[i] += take[i]
    assert at == lens
    assert float(np.abs(host(kept)[[0, 2, 4]]).max()) == 0.0


@pytest.mark.parametrize("H,G,d,e", [(4, 2, 20, 12), (3, 3, 7, 5), (6, 1, 64, 64), (2, 2, 128, 17), (2, 1, 130, 9), (2, 1, 300, 6), (1, 1, 512, 3)])
@pytest.mark.parametrize("ones", [False, True])
def test_weighted_sum_with_skip_or_normaliser(H, G, d, e, ones):
    """Decay and weight per token, in portions and token by token, states in slots of wider rows, a padding sequence; with
    `ones` the sum of the weighted keys read out beside it."""
    from braidinfer_amd import kernels as K
    rng = np.random.default_rng(H + d)
    T = 75
    q, k, v = f32(rng.standard_normal((T, G, d))), f32(rng.standard_normal((T, G, d)) / math.sqrt(d)), f32(rng.standard_normal((T, H, e)))
    gb = f32(np.concatenate([0.6 + 0.4 * rng.random((T, H)), rng.random((T, H)) * 2], axis=1))
    skip = f32(rng.standard_normal(H))
    want = P.state_space_sum(v, k, q, gb[:, :H], gb[:, H:])
    want_n = P.state_space_sum(np.ones((T, H, 1)), k, q, gb[:, :H], gb[:, H:])[..., 0]
    if not ones:
        want = want + skip[:, None] * v
    shape = K.glr_state_shape(H, d, e + ones)
    n = int(np.prod(shape))
    area = torch.zeros((4, n + 5), device="cuda")
    state = area[:, :n].view((4,) + shape)
    got, got_n, at = [], [], 0
    for take in (40, 2, 1, 1, 17, 14):
        rows = [np.concatenate([a[at:at + take].reshape(take, -1), np.ones((1, a[0].size))]) for a in (q, k, v)]
        wide = dev_f(np.concatenate([rows[0], rows[1], rows[2], np.zeros((take + 1, 3))], axis=1))
        o, no = torch.full((take + 1, H * e), 7.0, device="cuda"), torch.full((take + 1, H), 7.0, device="cuda")
        _, cu, slots = batch([take, 1], [2, -1])
        K.dr_scan(wide[:, :G * d], wide[:, G * d:2 * G * d], wide[:, 2 * G * d:2 * G * d + H * e], dev_f(np.concatenate([gb[at:at + take], np.ones((1, 2 * H))])),
                  None, o, state, cu, slots, 2, H, G, d, e, weighted=True, skip=None if ones else dev_f(skip), n_out=no if ones else None)
        got.append(host(o)[:take])
        got_n.append(host(no)[:take])
        assert float(np.abs(host(o)[take]).max()) == 0.0          # the padding row
        at += take
    scale = max(1.0, np.abs(want).max())
    assert np.abs(np.concatenate(got).reshape(T, H, e) - want).max() < 2e-5 * scale
    if ones:
        assert np.abs(np.concatenate(got_n) - want_n).max() < 2e-5 * max(1.0, np.abs(want_n).max())
    left = host(area)
    assert float(np.abs(left[[0, 1, 3]]).max()) == 0.0 and float(np.abs(left[2, n:]).max()) == 0.0


@pytest.mark.parametrize("H,G,d,e,ones,pieces", [(4, 2, 20, 12, False, 3), (2, 2, 64, 64, True, 5), (3, 1, 130, 9, True, 2), (2, 1, 16, 33, False, 16)])
def test_weighted_sum_in_pieces_behind_an_earlier_portion(H, G, d, e, ones, pieces):
    from braidinfer_amd import kernels as K
    from braidinfer_amd.parts.gated_recurrence import HGRN2
    rng = np.random.default_rng(d)
    first, lens = [9, 1], [150, 37]
    seqs = []
    for a, b in zip(first, lens):
        T = a + b
        q, k, v = f32(rng.standard_normal((T, G, d))), f32(rng.standard_normal((T, G, d)) / math.sqrt(d)), f32(rng.standard_normal((T, H, e)))
        gb = f32(np.concatenate([0.9 + 0.1 * rng.random((T, H)), rng.random((T, H))], axis=1))
        seqs.append((q, k, v, gb))
    skip = f32(rng.standard_normal(H))
    shape = K.glr_state_shape(H, d, e + ones)
    state = torch.zeros((3,) + tuple(shape), device="cuda")
    outs = []
    for part, pcs in ((0, 1), (1, pieces)):
        cut = [(slice(0, a) if part == 0 else slice(a, a + b)) for a, b in zip(first, lens)]
        n = [c.stop - c.start for c in cut]
        q, k, v, gb = (dev_f(np.concatenate([s[i][c].reshape(c.stop - c.start, -1) for s, c in zip(seqs, cut)])) for i in range(4))
        T = sum(n)
        o, no = torch.zeros((T, H * e), device="cuda"), torch.zeros((T, H), device="cuda")
        _, cu, slots = batch(n, [2, 0])
        more = dict(skip=None if ones else dev_f(skip), n_out=no if ones else None)
        if pcs == 1:
            K.dr_scan(q, k, v, gb, None, o, state, cu, slots, 2, H, G, d, e, weighted=True, **more)
        else:
            step = Step(T)
            step.extras, step.host_new, step.host_slots, step.tokens = {}, n, [2, 0], cu
            pcu, numbers = HGRN2._piece_arrays(step, pcs)
            K.dr_scan_pieces(q, k, v, None, o, state, slots, pcu, numbers, torch.zeros((2 * pcs,) + tuple(shape), device="cuda"), 2, pcs, H, d, e, G=G, gb=gb,
                             piece_decay=torch.zeros((2 * pcs, H), device="cuda"), **more)
        outs.append((host(o), host(no), n))
    for i, (q, k, v, gb) in enumerate(seqs):
        want = P.state_space_sum(v, k, q, gb[:, :H], gb[:, H:])
        want_n = P.state_space_sum(np.ones(v.shape[:2] + (1,)), k, q, gb[:, :H], gb[:, H:])[..., 0]
        if not ones:
            want = want + skip[:, None] * v
        lo = [0 if i == 0 else o[2][0] for o in outs]
        got = np.concatenate([o[0][l:l + o[2][i]] for o, l in zip(outs, lo)]).reshape(want.shape)
        assert np.abs(got - want).max() < 5e-5 * max(1.0, np.abs(want).max()), f"sequence {i}"
        if ones:
            got_n = np.concatenate([o[1][l:l + o[2][i]] for o, l in zip(outs, lo)])
            assert np.abs(got_n - want_n).max() < 5e-5 * max(1.0, np.abs(want_n).max())


@pytest.mark.parametrize("H,cap,shift", [(3, 15.0, 0.0), (5, 2.0, 3.0), (1, 15.0, -20.0), (2, 8.0, 20.0)])
def test_exponential_gates_over_a_running_maximum(H, cap, shift):
    """Portions shorter and longer than a wave's 64 and a workgroup's 1,024 tokens, beside a padding sequence; gates that
    saturate on both sides.  The running maximum starts at 0."""
    from braidinfer_amd import kernels as K
    rng = np.random.default_rng(H)
    T = 2300
    zi, zf = f32(rng.standard_normal((T, H)) * 4 + shift), f32(rng.standard_normal((T, H)) * 4 - shift)
    bi, bf_ = f32(rng.standard_normal(H)), f32(rng.standard_normal(H))
    i = cap * np.tanh((zi + bi) / cap)
    f = P.log_sigmoid(cap * np.tanh((zf + bf_) / cap))
    m, before, run = np.zeros((T, H)), np.zeros((T, H)), np.zeros(H)
    for t in range(T):
        before[t] = run
        run = m[t] = np.maximum(f[t] + run, i[t])
    keep, write = np.exp(f + before - m), np.exp(i - m)
    kept = torch.zeros((3, H + 2), device="cuda")
    at = 0
    for take in (1, 1, 2, 63, 64, 65, 1, 1030, 1, 1072):
        wide = dev_f(np.concatenate([np.concatenate([zi[at:at + take], zf[at:at + take], np.zeros((take, 1))], axis=1), np.zeros((1, 2 * H + 1))]))
        gb, mo = torch.zeros((take + 1, 2 * H), device="cuda"), torch.zeros((take + 1, H), device="cuda")
        _, cu, slots = batch([take, 1], [2, -1])
        K.exp_gates(wide[:, :H], wide[:, H:2 * H], dev_f(bi), dev_f(bf_), cap, kept[:, 1:1 + H], cu, slots, gb, mo, 2, single_tokens=take == 1)
        assert np.abs(host(mo)[:take] - m[at:at + take]).max() < 2e-5 * max(1.0, np.abs(m).max())
        assert np.abs(host(gb)[:take, :H] - keep[at:at + take]).max() < 3e-5 and np.abs(host(gb)[:take, H:] - write[at:at + take]).max() < 3e-5
        at += take
    assert at == T
    left = host(kept)
    assert float(np.abs(left[:2]).max()) == 0.0 and left[2, 0] == left[2, -1] == 0.0


@pytest.mark.parametrize("T,H,e", [(9, 3, 24), (9, 5, 7), (9, 4, 128), (9, 2, 512), (1030, 4, 512), (9, 1, 1100), (9, 2, 515), (9, 6, 1)])
@pytest.mark.parametrize("sigmoid", [False, True])
def test_gate_ahead_of_the_norm_and_the_normaliser(T, H, e, sigmoid):
    from braidinfer_amd import kernels as K
    rng = np.random.default_rng(e)
    eps = 1e-3
    o, w = f32(rng.standard_normal((T, H, e)) * 0.05), f32(1 + 0.2 * rng.standard_normal(H * e))
    wide = f32(rng.standard_normal((T, H * e + 4)) * 2)
    gate = wide[:, 4:].reshape(T, H, e)
    act = P.sigmoid(gate) if sigmoid else P.silu(gate)
    n, m = f32(rng.standard_normal((T, H)) * 3), f32(rng.standard_normal((T, H)) * 2)
    n[0, 0], m[0, 0] = 0.0, 12.0                          # exp(-m) decides
    q_mul = 0.3
    divided = o * q_mul / (np.maximum(np.abs(n * q_mul), np.exp(-m)) + 1e-6)[..., None]
    wh = w.reshape(H, e)
    for out, tol in ((torch.zeros((T, H * e), device="cuda"), 2e-5), (torch.zeros((T, H * e), dtype=torch.bfloat16, device="cuda"), 2e-2)):
        def check(want, **more):
            K.head_norm_gate(dev_f(o.reshape(T, -1)), dev_f(w), dev_f(wide)[:, 4:], out, H, e, eps, gate_sigmoid=sigmoid, **more)
            assert np.abs(host(out).reshape(T, H, e) - want).max() < tol * max(1.0, np.abs(want).max())
        check(P.rms_divide(o, eps) * wh * act)
        check(P.rms_divide(o * act, eps) * wh, gate_first=True)
        check(P.rms_divide(divided, eps) * wh * act, normaliser=(dev_f(n), dev_f(m), q_mul))


@pytest.mark.parametrize("H,G,d,e", [(4, 2, 16, 12), (3, 3, 7, 5), (6, 1, 64, 64), (2, 2, 128, 17), (2, 1, 130, 9), (2, 1, 300, 6)])
def test_delta_rule_with_decays_per_key_channel(H, G, d, e):
    from braidinfer_amd import kernels as K
    rng = np.random.default_rng(H + d)
    T = 61
    unit = lambda a: a / np.sqrt((a * a).sum(axis=-1, keepdims=True))
    q, k, v = f32(unit(rng.standard_normal((T, G, d)))), f32(unit(rng.standard_normal((T, G, d)))), f32(rng.standard_normal((T, H, e)))
    g, beta = f32(0.3 + 0.7 * rng.random((T, H, d))), f32(rng.random((T, H)))
    want = P.channel_delta_rule(q, k, v, g, beta)
    shape = K.glr_state_shape(H, d, e)
    state = torch.zeros((3,) + tuple(shape), device="cuda")
    got, at = [], 0
    for take in (30, 2, 1, 1, 16, 11):
        pad = lambda a: dev_f(np.concatenate([a[at:at + take].reshape(take, -1), np.ones((1, a[0].size))]))
        gb = torch.full((take + 1, 2 * H), float("nan"), device="cuda")          # the first half is not read
        gb[:, H:] = pad(beta)
        o = torch.full((take + 1, H * e), 7.0, device="cuda")
        _, cu, slots = batch([take, 1], [1, -1])
        K.dr_scan(pad(q), pad(k), pad(v), gb, None, o, state, cu, slots, 2, H, G, d, e, gc=pad(g))
        got.append(host(o)[:take])
        assert float(np.abs(host(o)[take]).max()) == 0.0
        at += take
    assert np.abs(np.concatenate(got).reshape(T, H, e) - want).max() < 2e-5 * max(1.0, np.abs(want).max())
    # a decay of its own for one channel alone: only that channel's rows of the state fade
    g1 = np.ones((2, H, d))
    g1[1, :, 0] = 0.0
    k1 = np.zeros((2, G, d))
    k1[0, :, 0] = k1[0, :, 1] = math.sqrt(0.5)
    s = torch.zeros((1,) + tuple(shape), device="cuda")
    o = torch.zeros((2, H * e), device="cuda")
    _, cu, slots = batch([2], [0])
    K.dr_scan(dev_f(np.zeros((2, G * d))), dev_f(k1.reshape(2, -1)), dev_f(v[:2].reshape(2, -1)), dev_f(np.ones((2, 2 * H))), None, o, s, cu, slots, 1, H, G,
              d, e, gc=dev_f(g1.reshape(2, -1)))
    S = host(K.glr_state_dense(s[0], H, d, e))
    assert np.abs(S[:, 0]).max() == 0.0 and np.abs(S[:, 1] - math.sqrt(0.5) * v[0]).max() < 1e-5


@pytest.mark.parametrize("G,H,d,e,n", [(2, 4, 16, 12, 4), (1, 1, 5, 9, 3), (3, 3, 64, 128, 2), (1, 2, 200, 6, 1), (2, 2, 12, 260, 5)])
def test_delta_rule_inputs_with_decays_per_key_channel(G, H, d, e, n):
    """Convolution, unit vectors, write strengths and decays from strided views, in portions of many, two and one token."""
    from braidinfer_amd import kernels as K
    rng = np.random.default_rng(d)
    T, C = 29, 2 * G * d + H * e
    raw, z = f32(rng.standard_normal((T, C + H + 8))), f32(rng.standard_normal((T, H * d + 4)) * 3)
    taps, a_log, dt_bias = f32(rng.standard_normal((C, n))), f32(rng.standard_normal(H)), f32(rng.standard_normal(H * d))
    y = P.short_convolution(raw[:, :C], taps)
    unit = lambda a: a / np.sqrt((a * a).sum(axis=-1, keepdims=True) + 1e-6)
    q, k = unit(y[:, :G * d].reshape(T, G, d)) * d ** -0.5, unit(y[:, G * d:2 * G * d].reshape(T, G, d))
    g = np.exp(-np.exp(a_log)[None, :, None] * P.softplus(z[:, :H * d] + dt_bias).reshape(T, H, d))
    want = (q.reshape(T, -1), k.reshape(T, -1), y[:, 2 * G * d:], P.sigmoid(raw[:, C:C + H]), g.reshape(T, -1))
    for vec in (True, False):
        kept = torch.zeros((3, max(1, (n - 1) * C)), device="cuda")
        at = 0
        for take in (7, 1, 1, 2, 1, 17):
            rows, zz = dev_f(raw[at:at + take]), dev_f(z[at:at + take])
            out = [torch.zeros((take, w), device="cuda") for w in (G * d, G * d, H * e, 2 * H, H * d)]
            sot, cu, slots = batch([take], [2])
            K.dr_conv_prepare(rows[:, :C + H], dev_f(taps), kept if n > 1 else None, dev_f(a_log), dev_f(dt_bias), sot, cu, slots, *out[:4], 1, G, H, d, e,
                              taps_t=dev_f(taps.T.copy()) if vec else None, decay=zz[:, :H * d], gc=out[4], single_tokens=take == 1)
            got = [host(out[0]), host(out[1]), host(out[2]), host(out[3])[:, H:], host(out[4])]
            for what, a, b in zip(("q", "k", "v", "beta", "decay"), got, want):
                assert np.abs(a - b[at:at + take]).max() < 2e-5, f"{what} at {at}"
            at += take


def test_choice_within_groups_by_softmax_scores():
    from braidinfer_amd import kernels as K
    rng = np.random.default_rng(12)
    for T, E, top, groups, keep in ((40, 12, 4, 4, 3), (30, 64, 8, 8, 4), (9, 6, 3, 2, 1), (9, 6, 2, 6, 2), (9, 8, 8, 2, 2), (20, 72, 5, 12, 3), (11, 130, 8, 65, 9),
                                    (3, 512, 64, 4, 1), (1, 4, 1, 1, 1), (33, 10, 2, 5, 5)):
        z = f32(rng.standard_normal((T, E)) * 2)
        z[:, 1] = z[:, 0]                                            # ties go to the lower number
        want_c, want_w = P.choose_experts(z, top, groups, keep)
        chosen, share = torch.zeros((T, top), dtype=torch.int32, device="cuda"), torch.zeros((T, top), device="cuda")
        K.route_softmax(dev_f(z), None, chosen, share, top, 1.0, groups, keep)
        got = chosen.cpu().numpy()
        same = (got == want_c).all(axis=1)
        assert same.mean() > 0.9, f"{E} experts in {groups} groups: {np.flatnonzero(~same)}"
        assert np.abs(host(share) - want_w)[same].max() < 1e-6


@pytest.mark.parametrize("H,G,d,e,rd", [(4, 2, 16, 24, 8), (3, 3, 10, 6, 10), (1, 1, 6, 20, 0), (8, 2, 64, 64, 32), (4, 4, 128, 96, 128)])
def test_attention_rows_with_biases_and_a_norm_per_head(H, G, d, e, rd):
    """Biases join before the norm of every head, neighbours turn behind it; queries, and keys and values in their pages."""
    from braidinfer_amd import kernels as K
    rng = np.random.default_rng(H * 7 + d)
    T, eps = 300, 1e-3
    width = H * d + G * (d + e)
    raw, bias = f32(rng.standard_normal((T, width)) * 0.05), f32(rng.standard_normal(width) * 0.05)
    qn, kn = f32(1 + 0.3 * rng.standard_normal(d)), f32(1 + 0.3 * rng.standard_normal(d))
    pos = np.arange(T) + 60
    x = raw + bias
    q = P.rms_divide(x[:, :H * d].reshape(T, H, d), eps) * qn
    k = P.rms_divide(x[:, H * d:(H + G) * d].reshape(T, G, d), eps) * kn
    v = x[:, (H + G) * d:].reshape(T, G, e)
    if rd:
        q, k = P.turn_neighbours(q, pos, rd, 100.0), P.turn_neighbours(k, pos, rd, 100.0)
    n_pages = -(-int(pos[-1] + 1) // 64)
    table = np.full((3, n_pages), -1, dtype=np.int32)
    table[1] = rng.permutation(n_pages + 3)[:n_pages]
    for dtype, tol in ((torch.float32, 1e-4), (torch.bfloat16, 1e-2)):
        unit = torch.zeros((n_pages + 3, G * 64 * (d + e)), dtype=dtype, device="cuda")
        got = []
        for lo, hi in ((0, 41), (41, 42), (42, T)):
            n = hi - lo
            cos = sin = None
            if rd:
                cos, sin = torch.zeros((n, rd // 2), device="cuda"), torch.zeros((n, rd // 2), device="cuda")
                K.rope_table(dev_i(pos[lo:hi]), dev_f([100.0 ** (-2 * i / rd) for i in range(rd // 2)]), cos, sin)
            qo = torch.full((n, H * d), 9.0, dtype=dtype, device="cuda")
            K.pwa_prepare(dev_f(raw[lo:hi]), dev_f(bias), dev_f(qn), dev_f(kn), eps, cos, sin, rd, dev_i(pos[lo:hi]), dev_i(np.zeros(n)), dev_i([1]),
                          dev_i(table), qo, unit, None, None, 0, H, G, d, e, 64, True, adjacent=True)
            got.append(host(qo))
        assert np.abs(np.concatenate(got).reshape(T, H, d) - q).max() < tol * max(1.0, np.abs(q).max())
        pages = host(unit)
        for t in range(T):
            pg = pages[table[1, pos[t] // 64]]
            assert np.abs(pg[:G * 64 * d].reshape(G, 64, d)[:, pos[t] % 64] - k[t]).max() < tol * max(1.0, np.abs(k).max()), f"keys of token {t}"
            assert np.abs(pg[G * 64 * d:].reshape(G, e, 64)[:, :, pos[t] % 64] - v[t]).max() < tol * max(1.0, np.abs(v).max()), f"values of token {t}"


def test_a_bias_behind_the_attention_reaches_every_kind_of_reader():
    """Added by the reader where it says so, by a kernel into residual rows and into rows a branch stores."""
    from braidinfer_amd.config import PartSpec
    from braidinfer_amd.parts import ResidualSink, build_part
    cfg = model(40, 60, 2, [par(2, 1, 8, 8, 5, None, (2, 8, 8, 1, 1, 2))])
    import braidinfer_amd as B
    spec = B.spec_of(B.config_from_dict(cfg))
    part = build_part("mixer", PartSpec("pooled_window_attention", spec.layers[0].mixer.params))
    from braidinfer_amd.parts import MixerContext, Runtime
    rng = np.random.default_rng(1)
    w = {s.name: bf(rng.standard_normal(s.shape) * 0.3) for s in part.weight_specs("")}
    part.load({n: dev_f(a) for n, a in w.items()}, "", Runtime(torch.device("cuda"), torch.float32))
    T = 6
    h = f32(rng.standard_normal((T, 40)))
    want = P.window_attention(h, w, "", cfg["layers"][0]["mixer"]["left"], 1e-5, np.arange(T))
    step = Step(T)
    step.position_data, step.positions, step.seq_of_token = {}, dev_i(np.arange(T)), dev_i(np.zeros(T))
    step.slots, step.cu_seqlens, step.ctx_lens, step.n_seqs, step.max_new = dev_i([0]), dev_i([0, T]), dev_i([T]), 1, T

    def ctx():
        unit = torch.zeros((1, 2, 1, 64 * 8), device="cuda")
        return MixerContext(unit=0, storage=unit, block_table=dev_i([[0]]), page_tokens=64)
    x = torch.ones((T, 40), device="cuda")
    part.forward(dev_f(h), x, step, ctx())
    assert np.abs(host(x) - 1 - want).max() < 1e-5
    y = torch.full((T, 40), 5.0, device="cuda")
    part.forward(dev_f(h), ResidualSink(y, None, overwrite=True), step, ctx())
    assert np.abs(host(y) - want).max() < 1e-5
    sink = ResidualSink(torch.full((T, 40), 5.0, device="cuda"), None, overwrite=True)
    sink.takes_bias = True
    part.forward(dev_f(h), sink, step, ctx())
    assert np.abs(host(sink.x) + host(sink.bias) - want).max() < 1e-5 and np.abs(host(sink.bias) - w["o.b"]).max() == 0.0


def loud_model(size):
    """A one-layer model in which token 0's query meets token 1's key with a score far above all others (in elements that
    are not rotated), and token 1's value moves the logits; the state-space side counts for nothing."""
    W = 48
    cfg = model(W, 60, 2, [par(2, 1, 16, 16, size, (8, 10000.0), (2, 4, 4, 1, 1, 2), scales=(1.0, 0.0), scale=1.0)])
    w = P.random_weights(cfg, 31, gain=0.3)
    quiet = {"l0.norm1": np.ones(W), "l0.norm1.b": np.zeros(W), "l0.norm1.alpha": 0.25, "final.norm": np.ones(W), "final.norm.b": np.zeros(W),
             "final.norm.alpha": 0.25, "l0.hc1.in": [0.5, 0.5], "l0.hc1.out": [4.0, 4.0], "l0.hc1.mix": np.eye(2)}
    w.update({n: bf(a) for n, a in quiet.items()})
    emb = w["embed"] * 0.5
    emb[:, :2] = 0.0
    emb[0, 0] = emb[1, 1] = 12.0                         # element 0 marks the asking token, element 1 the loud one
    w["embed"] = emb
    p = "l0.mix.left."
    for n in ("q", "k"):
        w[p + n][:, :2] = 0.0
        w[p + n + ".b"][:] = 0.0
        w[p + n + ".norm"][:] = 1.0
    w[p + "q"][12, 0] = w[p + "q"][16 + 12, 0] = 30.0    # element 12 lies behind the rotated ones
    w[p + "k"][12, 1] = 30.0
    w[p + "v"][:, 1] = 2.0
    for n in list(w):
        w[n] = bf(w[n])
    return cfg, w


@pytest.mark.parametrize("size", [75, 64, 65, 1, 128, None])
def test_a_loud_key_at_every_edge(size, tmp_path):
    """One key whose score stands out just inside and just outside the window, at page borders, at the sequence's first
    token and hundreds of tokens away; asked for in a prompt, behind a portion and by a single token."""
    import braidinfer_amd as B
    cfg, w = loud_model(size)
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
                assert err < tol, f"{size} {dtype}: the query at {p} and key {j} ({'seen' if seen else 'unseen'}), portions {portions}: {err:.3g}"
        del eng


def remembering_model(kind):
    """A one-layer model whose recurrent mixer forgets next to nothing, with weights that let an early token show far away."""
    W = 48
    layer = {"state_space": par(2, 1, 8, 8, 3, None, (4, 12, 16, 2, 2, 4), scales=(0.0, 1.0)), "mlstm": mls(3, 12, 16, 15.0),
             "channel_delta": cdr(4, 2, 12, 16, 4)}[kind]
    cfg = model(W, 60, 2, [layer])
    w = P.random_weights(cfg, 77, gain=0.8)
    if kind == "mlstm":
        w["l0.mix.f.b"][:] = 12.0                        # log forget gates of about -1e-5
        w["l0.mix.f"][:] = 0.0
    else:
        p = "l0.mix." + ("right." if kind == "state_space" else "")
        w[p + "A_log"][:] = -7.0                         # decays of about exp(-1e-3)
    w["l0.hc1.out"][:] = 3.0
    for n in list(w):
        w[n] = bf(w[n])
    return cfg, w


@pytest.mark.parametrize("kind", ["state_space", "mlstm", "channel_delta"])
def test_a_token_remembered_from_far_away(kind, tmp_path):
    """The state, not a window, carries it: another first token, another token at a portion's border, hundreds of tokens
    back, shows in the logits, whole, in portions, token by token and beside another request whose slot was just used."""
    import braidinfer_amd as B
    cfg, w = remembering_model(kind)
    folder = str(tmp_path / "m")
    P.write_model(folder, cfg, w)
    T = 260
    base = tokens_of(cfg, T, 6)
    for dtype, tol in (("float32", 2e-4), ("bfloat16", 0.12)):
        eng = B.Engine.from_folder(folder, dtype=dtype, max_tokens=1024, n_slots=2)
        want0 = P.forward(cfg, w, base)
        for j in (0, 1, 63, 64):
            toks = list(base)
            toks[j] = (toks[j] + 17) % cfg["vocab"]
            want = P.forward(cfg, w, toks)
            moved = np.sqrt(((want - want0) ** 2).mean(axis=1))[-20:].min() / want.std()
            assert moved > 2e-3, f"token {j} is forgotten: {moved}"
            for portions in ([T], [64, T - 64], [63, 2, 100] + [1] * (T - 165)):
                got = run(eng, toks, portions)
                err = np.sqrt(((got - want) ** 2).mean(axis=1)) / want.std()
                assert err.max() < tol, f"{kind} {dtype} token {j} {portions[:3]}: {err.max():.3g} at {err.argmax()}"
        del eng


# ------------------------------------------------------------ whole models -----------
@pytest.mark.parametrize("name", list(CONFIGS))
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_whole_prompt_against_plain(folders, engines, name, dtype):
    _, cfg, w = folders[(name, dtype)]
    toks = tokens_of(cfg, 150, 1)
    want = plain(name, dtype, cfg, w, toks)
    close(run(engines(name, dtype), toks, [150]), want, dtype, f"{name} {dtype}", rounded(cfg, w, toks, dtype))
    close(run(engines(name, dtype), toks[:1], [1]), want[:1], dtype, "a sequence of one token", rounded(cfg, w, toks[:1], dtype))
    close(run(engines(name, dtype), toks[:3], [1, 1, 1]), want[:3], dtype, "the first tokens one by one", rounded(cfg, w, toks[:3], dtype))
    close(run(engines(name, dtype), toks[:5], [2, 3]), want[:5], dtype, "the first tokens in two portions", rounded(cfg, w, toks[:5], dtype))


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
    assert len(layers) == len(cfg["layers"])
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
        close(got, want, dtype, f"{name} {dtype} {portions[:4]}", rounded(cfg, w, toks, dtype))
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
        close(g, plain(name, dtype, cfg, w, p)[:len(g)], dtype, f"request {i} of the batch", rounded(cfg, w, p, dtype))


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
    """Requests come and go through a cache of few pages and two slots: what a returned page or slot held never shows, the
    windows' pages go back, and every page comes back."""
    import braidinfer_amd as B
    folder, cfg, w = folders[("a", "float32")]
    eng = B.Engine.from_folder(folder, dtype="float32", max_tokens=448, max_seq_len=448, n_slots=2)
    free_before = [g.pool.free_count for g in eng.cache.groups]
    assert sorted(eng.cache.group_of_unit) == [1, 3]                   # the parallel layers' attention; the others keep state only
    for r in range(5):
        toks = tokens_of(cfg, 120 + 67 * r, 50 + r)
        close(run(eng, toks, [len(toks) - 10] + [1] * 10), P.forward(cfg, w, toks), "float32", f"request {r}")
    assert [g.pool.free_count for g in eng.cache.groups] == free_before
    toks = tokens_of(cfg, 400, 77)
    s = eng.alloc_slot()
    got = [eng.step([B.StepEntry(s, toks[:380], [379])]).cpu().numpy()]
    held = lambda u: [i for i, p in enumerate(eng.cache.unit_group(u).pages[s]) if p >= 0]
    assert held(1) == [5] and held(3) == [4, 5]
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
        close(run(engines(name, dtype), toks, [30] + [1] * 300), plain(name, dtype, cfg, w, toks), dtype, f"{name} {dtype}",
              rounded(cfg, w, toks, dtype))


def test_a_long_prompt(folders, engines):
    for dtype in ("float32", "bfloat16"):
        _, cfg, w = folders[("c", dtype)]
        toks = tokens_of(cfg, 700, 8)
        want = plain("c", dtype, cfg, w, toks)
        close(run(engines("c", dtype), toks, [700]), want, dtype, f"whole {dtype}")
        close(run(engines("c", dtype), toks, [100, 600]), want, dtype, f"behind a portion {dtype}")


def drawn_configuration(seed):
    """A configuration drawn at random: any order of layers, head counts and widths from lists that hold odd ones and such
    that the matrix-core kernels take, any window, streams and groups, keys left out."""
    rng = np.random.default_rng(seed)
    pick = lambda xs: xs[int(rng.integers(len(xs)))]

    def heads():
        H = pick([1, 2, 3, 4, 6, 8, 12])
        return H, pick([g for g in (1, 2, 3, 4, 6, 8, 12) if H % g == 0])

    def mlp():
        r = rng.random()
        if r < 0.15:
            return None
        if r < 0.5:
            return dense(pick([8, 21, 40, 64]), pick([0.5, 1.0, 7.0]))
        E = pick([1, 2, 4, 6, 8, 12, 16])
        count = pick([g for g in (1, 2, 3, 4, 8) if E % g == 0])
        keep = int(rng.integers(1, count + 1))
        top = pick([t for t in (1, 2, 3, 4, 8) if t <= keep * (E // count)])
        return moe(pick([8, 16, 20, 40]), E, top, (count, keep) if count > 1 or rng.random() < 0.5 else None)
    layers = []
    for _ in range(int(rng.integers(2, 6))):
        kind = pick(["parallel", "mlstm", "channel_delta"])
        H, G = heads()
        if kind == "parallel":
            d = pick([6, 8, 12, 16, 24, 32, 64])
            rot = (pick([r for r in (2, 4, 8, 12, 16, 32, 64) if r <= d]), pick([100.0, 10000.0, 1e6])) if rng.random() < 0.85 else None
            h2, g2 = heads()
            e2 = pick([3, 4, 8, 12, 32])
            parts = pick([p for p in (1, 2, 3, 4, 6, 8) if h2 * e2 % p == 0])
            layers.append(par(H, G, d, pick([None, 8, 10, 16, 32, 64]), pick([None, 1, 7, 33, 64, 100]), rot,
                              (h2, e2, pick([3, 8, 16, 40, 130]), g2, parts, pick([1, 2, 3, 4, 7])), (pick([0.5, 1.0, -0.7]), pick([0.3, 1.0, 1.4])), mlp=mlp()))
        elif kind == "mlstm":
            layers.append(mls(H, pick([3, 8, 16, 40, 64]), pick([1, 4, 8, 15, 16, 32]), pick([1.0, 6.0, 15.0]), mlp=mlp()))
        else:
            layers.append(cdr(H, G, pick([3, 8, 16, 40, 64]), pick([4, 8, 15, 32]), pick([1, 2, 3, 4]), mlp=mlp()))
    return model(pick([32, 48, 50, 64, 80]), int(rng.integers(40, 300)), pick([1, 2, 2, 3, 4, 6]), layers, eps=pick([1e-6, 1e-5, 1e-3])), \
        (pick([1, 4, 9, 16]), pick([1, 3, 8, 24]))


@pytest.mark.parametrize("seed", range(16))
def test_configurations_drawn_at_random(seed, tmp_path):
    """Whole, in portions and token by token in float32 against the plain implementation; bfloat16 whole and decoded."""
    import braidinfer_amd as B
    cfg, ranks = drawn_configuration(5000 + seed)
    what = f"seed {seed}: {json.dumps(cfg)}"
    toks = tokens_of(cfg, 110, seed)
    other = tokens_of(cfg, 45, seed + 50)
    folder = str(tmp_path / "m")
    w = P.random_weights(cfg, seed=seed, gain=0.9, ranks=ranks)
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
    w = P.random_weights(cfg, seed=seed, gain=0.9, ranks=ranks, router_spread=0.5)
    P.write_model(folder, cfg, w)
    eng = B.Engine.from_folder(folder, dtype="bfloat16", max_tokens=512)
    close(run(eng, toks, [60] + [1] * 50), P.forward(cfg, w, toks), "bfloat16", what + " bfloat16", rounded(cfg, w, toks, "bfloat16"))


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


def test_the_command_line_generates_from_a_tuzisun_folder(folders):
    """`bin/generate` on a Tuzisun folder: the model class by config.json, greedy tokens as the plain implementation's; a
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
    cfg = B.any_preset("tuzisun-tiny")
    folder = B.Engine.write_random_folder(str(tmp_path / "m"), cfg, seed=3, std=0.1, vector_jitter=0.3)
    pc, pw = P.read_model(folder)
    toks = tokens_of(pc, 120, 4)
    eng = B.Engine.from_folder(folder, dtype="float32", max_tokens=512)
    close(run(eng, toks, [90] + [1] * 30), P.forward(pc, pw, toks), "float32", "preset")


def test_replay_of_given_tokens_through_the_command(folders, tmp_path):
    """`bin/trace_run` as a child process on a Tuzisun folder: requests whole, with their last tokens one by one, and two
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
