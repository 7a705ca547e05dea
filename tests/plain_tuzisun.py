"""A plain, slow implementation of the Tuzisun design in NumPy float64, one function per
mechanism, written from the design's equations.  It shares no code with the library: the
tests hold the engine against it.

Notation: a sequence's tokens are rows; positions count from 0.  `cfg` is the model's
configuration as a dict (the keys of its config.json), `w` maps tensor names to float arrays.
The residual is a set of streams x_1 .. x_s; every half of a layer reads one weighted sum of
them and writes its output back into all of them.
"""
from __future__ import annotations

import json
import math
import os
import struct

import numpy as np

ALPHA = 1.702


# ------------------------------------------------------------------ mechanisms ------
def dynamic_tanh(x, w, name):
    """tanh(alpha x) weight + bias, element by element."""
    return np.tanh(w[name + ".alpha"] * x) * w[name] + w[name + ".b"]


def rms_divide(x, eps):
    """x / sqrt(mean(x^2) + eps) over the last axis."""
    return x / np.sqrt((x * x).mean(axis=-1, keepdims=True) + eps)


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def silu(z):
    return z * sigmoid(z)


def softplus(z):
    return np.maximum(z, 0.0) + np.log1p(np.exp(-np.abs(z)))


def log_sigmoid(z):
    return -softplus(-z)


def softmax(z):
    p = np.exp(z - z.max(axis=-1, keepdims=True))
    return p / p.sum(axis=-1, keepdims=True)


def turn_neighbours(x, positions, dims, base):
    """x [T, heads, d]: elements 2i and 2i + 1 of the first `dims` of every head turned by position * base^(-2i/dims)."""
    y = np.array(x, dtype=np.float64)
    for i in range(dims // 2):
        ang = np.asarray(positions, dtype=np.float64)[:, None] * base ** (-2.0 * i / dims)
        u, v = x[..., 2 * i], x[..., 2 * i + 1]
        y[..., 2 * i] = u * np.cos(ang) - v * np.sin(ang)
        y[..., 2 * i + 1] = v * np.cos(ang) + u * np.sin(ang)
    return y


def window(T, size):
    """Key j is seen by query i when 0 <= i - j < size (size None: every j <= i)."""
    d = np.arange(T)[:, None] - np.arange(T)[None, :]
    return (d >= 0) & (d < (T if size is None else size))


def softmax_attention(q, k, v, scale, visible):
    """q [T, H, d], k [T, G, d], v [T, G, e] -> [T, H, e]; query head h reads key/value head h // (H / G)."""
    T, H, _ = q.shape
    G = k.shape[1]
    out = np.zeros((T, H, v.shape[2]))
    for h in range(H):
        g = h // (H // G)
        s = np.where(visible, (q[:, h] @ k[:, g].T) * scale, -np.inf)
        out[:, h] = softmax(s) @ v[:, g]
    return out


def short_convolution(x, taps, bias=None):
    """x [T, C], taps [C, n] (the last column multiplies the current token), zeros before the start, then silu."""
    T, n = x.shape[0], taps.shape[1]
    y = np.zeros_like(x)
    for j in range(n):
        back = n - 1 - j
        if back < T:
            y[back:] += x[:T - back] * taps[:, j]
    return silu(y if bias is None else y + bias)


def state_space_sum(x, B, C, decay, step):
    """Per head S_t = decay_t S_(t-1) + step_t B_t x_t^T, y_t = S_t^T C_t.  x [T, H, e], B and C [T, G, N], decay and
    step [T, H]; head h reads group h // (H / G)."""
    T, H, e = x.shape
    G, N = B.shape[1:]
    y = np.zeros((T, H, e))
    for h in range(H):
        S, g = np.zeros((N, e)), h // (H // G)
        for t in range(T):
            S = decay[t, h] * S + step[t, h] * np.outer(B[t, g], x[t, h])
            y[t, h] = S.T @ C[t, g]
    return y


def matrix_memory(q, k, v, i, f):
    """Exponential input gates and sigmoid forget gates (their logarithms i, f [T, H]) over an outer-product memory and
    its normaliser, both kept relative to exp(m).  q, k [T, H, d], v [T, H, e] -> [T, H, e]."""
    T, H, d = q.shape
    out = np.zeros((T, H, v.shape[2]))
    for h in range(H):
        S, n, m = np.zeros((d, v.shape[2])), np.zeros(d), 0.0
        for t in range(T):
            new = max(f[t, h] + m, i[t, h])
            keep, write = math.exp(f[t, h] + m - new), math.exp(i[t, h] - new)
            S = keep * S + write * np.outer(k[t, h], v[t, h])
            n = keep * n + write * k[t, h]
            m = new
            out[t, h] = S.T @ q[t, h] / (max(abs(float(n @ q[t, h])), math.exp(-m)) + 1e-6)
    return out


def channel_delta_rule(q, k, v, g, beta):
    """Decay of the key channels, correction of what the key reads, write, read: q, k [T, G, d], v [T, H, e],
    g [T, H, d], beta [T, H] -> [T, H, e]; head h reads q/k head h // (H / G)."""
    T, H, e = v.shape
    G, d = q.shape[1:]
    out = np.zeros((T, H, e))
    for h in range(H):
        S, gh = np.zeros((d, e)), h // (H // G)
        for t in range(T):
            S = g[t, h][:, None] * S
            u = beta[t, h] * (v[t, h] - S.T @ k[t, gh])
            S = S + np.outer(k[t, gh], u)
            out[t, h] = S.T @ q[t, gh]
    return out


def clamped_unit(h, gate, up, down, limit):
    """g sigmoid(1.702 g) (u + 1) through `down`, g bounded from above and u on both sides."""
    g = np.minimum(h @ gate.T, limit)
    u = np.clip(h @ up.T, -limit, limit)
    return (g * sigmoid(ALPHA * g) * (u + 1.0)) @ down.T


def choose_experts(z, top, groups=1, keep=1):
    """z [T, E] router logits.  s = softmax(z); the experts form `groups` runs of neighbours, a run scores its largest s,
    and the `top` largest s within the `keep` best runs are chosen (ties to the lower number), their weights s as it is."""
    s = softmax(z)
    T, E = s.shape
    c = s.copy()
    if groups > 1:
        runs = s.reshape(T, groups, E // groups).max(axis=2)
        best = np.argsort(-runs, axis=1, kind="stable")[:, :keep]
        allowed = np.zeros((T, groups), dtype=bool)
        np.put_along_axis(allowed, best, True, axis=1)
        c = np.where(np.repeat(allowed, E // groups, axis=1), s, -np.inf)
    chosen = np.argsort(-c, axis=1, kind="stable")[:, :top]
    return chosen, np.take_along_axis(s, chosen, axis=1)


# ------------------------------------------------------------------ mixers ----------
def window_attention(h, w, p, m, eps, positions):
    """Grouped heads in a sliding window, biases on every projection, a norm per head of queries and keys, neighbouring
    elements turned."""
    T = h.shape[0]
    H, G, d, e = m["heads"], m.get("kv_heads", m["heads"]), m["dim"], m.get("vdim", m["dim"])
    q = (h @ w[p + "q"].T + w[p + "q.b"]).reshape(T, H, d)
    k = (h @ w[p + "k"].T + w[p + "k.b"]).reshape(T, G, d)
    v = (h @ w[p + "v"].T + w[p + "v.b"]).reshape(T, G, e)
    q, k = rms_divide(q, eps) * w[p + "q.norm"], rms_divide(k, eps) * w[p + "k.norm"]
    rot = m.get("rot")
    if rot:
        q = turn_neighbours(q, positions, rot["dims"], rot["base"])
        k = turn_neighbours(k, positions, rot["dims"], rot["base"])
    o = softmax_attention(q, k, v, m["scale"], window(T, (m.get("mask") or {}).get("size")))
    return o.reshape(T, H * e) @ w[p + "o"].T + w[p + "o.b"]


def state_space_mixer(h, w, p, m, eps):
    """Mamba-2: gate | inputs | B | C | step sizes in one projection; convolution, state, gate, norm in equal parts."""
    T = h.shape[0]
    H, e, N, G, parts = m["heads"], m["vdim"], m["state"], m.get("groups", 1), m.get("norm_groups", 1)
    inner = H * e
    rows = h @ w[p + "in"].T
    z, xbc, dt = rows[:, :inner], rows[:, inner:2 * inner + 2 * G * N], rows[:, 2 * inner + 2 * G * N:]
    xbc = short_convolution(xbc, w[p + "conv"], w[p + "conv.b"])
    x = xbc[:, :inner].reshape(T, H, e)
    B, C = xbc[:, inner:inner + G * N].reshape(T, G, N), xbc[:, inner + G * N:].reshape(T, G, N)
    dt = softplus(dt + w[p + "dt_bias"])
    y = state_space_sum(x, B, C, np.exp(-np.exp(w[p + "A_log"]) * dt), dt) + w[p + "D"][:, None] * x
    y = (y.reshape(T, inner) * silu(z)).reshape(T, parts, inner // parts)
    return (rms_divide(y, eps).reshape(T, inner) * w[p + "norm"]) @ w[p + "o"].T


def parallel_mixer(h, w, p, m, eps, positions):
    return (m.get("left_scale", 1.0) * window_attention(h, w, p + "left.", m["left"], eps, positions)
            + m.get("right_scale", 1.0) * state_space_mixer(h, w, p + "right.", m["right"], eps))


def mlstm_gates(h, w, p, cap):
    """Logarithms of the input and the forget gates, both soft-bounded by `cap`."""
    i = cap * np.tanh((h @ w[p + "i"].T + w[p + "i.b"]) / cap)
    f = log_sigmoid(cap * np.tanh((h @ w[p + "f"].T + w[p + "f.b"]) / cap))
    return i, f


def mlstm_mixer(h, w, p, m, eps, positions):
    T = h.shape[0]
    H, d, e = m["heads"], m["dim"], m.get("vdim", m["dim"])
    q = (h @ w[p + "q"].T).reshape(T, H, d) * d ** -0.5
    k, v = (h @ w[p + "k"].T).reshape(T, H, d), (h @ w[p + "v"].T).reshape(T, H, e)
    i, f = mlstm_gates(h, w, p, m["gate_cap"])
    o = rms_divide(matrix_memory(q, k, v, i, f), eps).reshape(T, H * e)
    return (o * w[p + "norm"] * sigmoid(h @ w[p + "g"].T)) @ w[p + "o"].T


def channel_delta_mixer(h, w, p, m, eps, positions):
    T = h.shape[0]
    H, G, d, e = m["heads"], m.get("kv_heads", m["heads"]), m["dim"], m.get("vdim", m["dim"])
    q = short_convolution(h @ w[p + "q"].T, w[p + "q.conv"]).reshape(T, G, d)
    k = short_convolution(h @ w[p + "k"].T, w[p + "k.conv"]).reshape(T, G, d)
    v = short_convolution(h @ w[p + "v"].T, w[p + "v.conv"]).reshape(T, H, e)
    q = q / np.sqrt((q * q).sum(axis=-1, keepdims=True) + 1e-6) * d ** -0.5
    k = k / np.sqrt((k * k).sum(axis=-1, keepdims=True) + 1e-6)
    beta = sigmoid(h @ w[p + "b"].T)
    step = softplus((h @ w[p + "a1"].T) @ w[p + "a2"].T + w[p + "dt_bias"].reshape(-1)).reshape(T, H, d)
    g = np.exp(-np.exp(w[p + "A_log"])[None, :, None] * step)
    o = rms_divide(channel_delta_rule(q, k, v, g, beta), eps) * w[p + "norm"]
    gate = sigmoid((h @ w[p + "g1"].T) @ w[p + "g2"].T)
    return (o.reshape(T, H * e) * gate) @ w[p + "o"].T


MIXERS = {"parallel": parallel_mixer, "mlstm": mlstm_mixer, "channel_delta": channel_delta_mixer}


# ------------------------------------------------------------------ feed-forward ----
def feed_forward(h, w, p, f):
    if f["kind"] == "dense":
        return clamped_unit(h, w[p + "gate"], w[p + "up"], w[p + "down"], f["limit"])
    r = f["router"]
    groups = r.get("groups") or {}
    chosen, weights = choose_experts(h @ w[p + "router"].T, r["top"], groups.get("count", 1), groups.get("keep", 1))
    out = np.zeros_like(h)
    for t in range(h.shape[0]):
        for j, share in zip(chosen[t], weights[t]):
            q = p + "e%d." % j
            out[t] += share * (w[q + "down"] @ (silu(w[q + "gate"] @ h[t]) * (w[q + "up"] @ h[t])))
    return out


# ------------------------------------------------------------------ the model -------
def connected_half(streams, half, w, c, norm):
    """streams [s, T, width].  u = sum_s in[s] x_s; y = half(norm(u)); x_t <- sum_s mix[s, t] x_s + out[t] y, all t at once."""
    u = np.tensordot(w[c + "in"], streams, axes=(0, 0))
    y = half(norm(u))
    return np.tensordot(w[c + "mix"].T, streams, axes=(1, 0)) + w[c + "out"][:, None, None] * y[None]


def forward(cfg, w, tokens, return_layers=False, round_inputs=False):
    """Logits [T, vocab] of one sequence from position 0 (and the sum of the streams after every layer).  `round_inputs`
    rounds what every half and the head read to bfloat16 values: how far that alone moves the logits says what a model is
    worth in bfloat16."""
    point = (lambda x: to_bf16_values(x)) if round_inputs else (lambda x: x)
    eps = cfg["norm"]["eps"]
    x = np.repeat(w["embed"][np.asarray(tokens)][None], cfg.get("streams", 1), axis=0)
    positions = np.arange(len(tokens))
    rows = []
    for i, layer in enumerate(cfg["layers"]):
        p = "l%d." % i
        x = connected_half(x, lambda h: MIXERS[layer["type"]](h, w, p + "mix.", layer["mixer"], eps, positions), w, p + "hc1.",
                           lambda u: point(dynamic_tanh(u, w, p + "norm1")))
        if layer.get("mlp"):
            x = connected_half(x, lambda h: feed_forward(h, w, p + "mlp.", layer["mlp"]), w, p + "hc2.",
                               lambda u: point(dynamic_tanh(u, w, p + "norm2")))
        rows.append(x.sum(axis=0))
    logits = point(dynamic_tanh(x.sum(axis=0), w, "final.norm")) @ w["embed"].T
    return (logits, np.stack(rows)) if return_layers else logits


def greedy(cfg, w, prompt, n):
    tokens = list(prompt)
    for _ in range(n):
        tokens.append(int(np.argmax(forward(cfg, w, tokens)[-1])))
    return tokens[len(prompt):]


# ------------------------------------------------------------------ weights ---------
def tensor_shapes(cfg, ranks=(5, 7)):
    """name -> shape of every tensor of a model of this configuration.  `ranks`: the inner widths of the decay's and the
    gate's low-rank projections, which the tensors alone give."""
    W, V, s = cfg["width"], cfg["vocab"], cfg.get("streams", 1)
    out = {"embed": (V, W)}

    def norm(name):
        out[name], out[name + ".b"], out[name + ".alpha"] = (W,), (W,), ()

    for i, layer in enumerate(cfg["layers"]):
        p, m, f = "l%d." % i, layer["mixer"], layer.get("mlp")
        for half in ("1", "2") if f else ("1",):
            norm(p + "norm" + half)
            out[p + "hc%s.in" % half] = out[p + "hc%s.out" % half] = (s,)
            out[p + "hc%s.mix" % half] = (s, s)
        q = p + "mix."
        if layer["type"] == "parallel":
            a, q = m["left"], p + "mix.left."
            H, G, d, e = a["heads"], a.get("kv_heads", a["heads"]), a["dim"], a.get("vdim", a["dim"])
            for n, size in (("q", H * d), ("k", G * d), ("v", G * e)):
                out[q + n], out[q + n + ".b"] = (size, W), (size,)
            out[q + "q.norm"] = out[q + "k.norm"] = (d,)
            out[q + "o"], out[q + "o.b"] = (W, H * e), (W,)
            a, q = m["right"], p + "mix.right."
            inner, bc = a["heads"] * a["vdim"], 2 * a.get("groups", 1) * a["state"]
            out[q + "in"] = (2 * inner + bc + a["heads"], W)
            out[q + "conv"], out[q + "conv.b"] = (inner + bc, a["conv"]), (inner + bc,)
            out[q + "dt_bias"] = out[q + "A_log"] = out[q + "D"] = (a["heads"],)
            out[q + "norm"], out[q + "o"] = (inner,), (W, inner)
        elif layer["type"] == "mlstm":
            H, d, e = m["heads"], m["dim"], m.get("vdim", m["dim"])
            out[q + "q"] = out[q + "k"] = (H * d, W)
            out[q + "v"] = out[q + "g"] = (H * e, W)
            out[q + "i"] = out[q + "f"] = (H, W)
            out[q + "i.b"] = out[q + "f.b"] = (H,)
            out[q + "norm"], out[q + "o"] = (H * e,), (W, H * e)
        else:
            H, G, d, e, n = m["heads"], m.get("kv_heads", m["heads"]), m["dim"], m.get("vdim", m["dim"]), m["conv"]
            for x, size in (("q", G * d), ("k", G * d), ("v", H * e)):
                out[q + x], out[q + x + ".conv"] = (size, W), (size, n)
            out[q + "b"], out[q + "A_log"], out[q + "dt_bias"] = (H, W), (H,), (H * d,)
            out[q + "a1"], out[q + "a2"] = (ranks[0], W), (H * d, ranks[0])
            out[q + "g1"], out[q + "g2"] = (ranks[1], W), (H * e, ranks[1])
            out[q + "norm"], out[q + "o"] = (e,), (W, H * e)
        if not f:
            continue
        q = p + "mlp."
        if f["kind"] == "dense":
            out[q + "gate"] = out[q + "up"] = (f["ff"], W)
            out[q + "down"] = (W, f["ff"])
            continue
        for j in range(f["router"]["experts"]):
            n = f["expert"]["ff"]
            out[q + "e%d.gate" % j], out[q + "e%d.up" % j], out[q + "e%d.down" % j] = (n, W), (n, W), (W, n)
        out[q + "router"] = (f["router"]["experts"], W)
    norm("final.norm")
    return out


def to_bf16_values(a):
    """Round float64 values to the nearest bfloat16 (ties to even), returned as float64."""
    a32 = np.asarray(a, dtype=np.float32)
    u = a32.reshape(-1).view(np.uint32).astype(np.uint64)
    u = ((u + 0x7FFF + ((u >> 16) & 1)) >> 16) << 16
    return u.astype(np.uint32).view(np.float32).astype(np.float64).reshape(a32.shape)


def random_weights(cfg, seed, gain=1.0, ranks=(5, 7), router_spread=None):
    """Weights that keep every activation of order one, already rounded to bfloat16.  `gain` sizes the matrices.
    `router_spread`: the first channel of every feed-forward's input is 1 whatever the token, and the routers read it with
    weights that far apart and the other channels with small ones, so that a bfloat16 run chooses as the float64 run does."""
    rng = np.random.default_rng(seed)
    w = {}
    s = cfg.get("streams", 1)
    for name, shape in tensor_shapes(cfg, ranks).items():
        tail = name.split(".")[-1]
        if tail == "alpha":
            a = np.array(0.5 + 0.4 * rng.random())
        elif name.endswith("norm.b") or name.endswith("norm1.b") or name.endswith("norm2.b"):
            a = 0.2 * rng.standard_normal(shape)
        elif "norm" in tail:
            a = 1.0 + 0.2 * rng.standard_normal(shape)
        elif ".hc" in name and tail == "in":
            a = (1.0 + 0.4 * rng.standard_normal(shape)) / s
        elif ".hc" in name and tail == "out":
            a = 0.7 + 0.3 * rng.standard_normal(shape)
        elif ".hc" in name:
            a = 0.7 * np.eye(s) + (0.3 + 0.3 * rng.standard_normal(shape)) / s
        elif tail == "A_log":
            a = np.log(0.05 + 0.6 * rng.random(shape))
        elif tail == "dt_bias":
            a = -1.0 + rng.standard_normal(shape)
        elif tail == "conv" or name.endswith("conv.b"):
            a = rng.standard_normal(shape) * 0.5
        elif tail == "D":
            a = 1.0 + 0.3 * rng.standard_normal(shape)
        elif name.endswith(".f.b"):
            a = 2.0 + rng.standard_normal(shape)
        elif tail == "b" and len(shape) == 1:
            a = 0.3 * rng.standard_normal(shape)
        elif name == "embed":
            a = rng.standard_normal(shape)
        elif tail == "router" and router_spread is not None:
            a = rng.standard_normal(shape) * (0.1 / math.sqrt(shape[-1]))
            a[:, 0] = router_spread * rng.permutation(shape[0])
        else:
            a = rng.standard_normal(shape) * (1.5 * gain / math.sqrt(shape[-1]))
        w[name] = to_bf16_values(a)
        if router_spread is not None and ".norm2" in name and shape:
            w[name][0] = 1.0 if tail == "b" else 0.0
    return w


def write_safetensors(path, w, dtype="bfloat16"):
    """Write `w` as one safetensors file of bfloat16 (or float32) tensors."""
    header, blobs, at = {}, [], 0
    for name, a in w.items():
        a32 = np.asarray(a, dtype=np.float32)
        shape = list(a32.shape)
        a32 = np.ascontiguousarray(a32).reshape(-1)
        if dtype == "bfloat16":
            blob = (a32.view(np.uint32) >> 16).astype(np.uint16).tobytes()
            tag = "BF16"
        else:
            blob, tag = a32.tobytes(), "F32"
        header[name] = {"dtype": tag, "shape": shape, "data_offsets": [at, at + len(blob)]}
        blobs.append(blob)
        at += len(blob)
    text = json.dumps(header, separators=(",", ":")).encode()
    text += b" " * (-len(text) % 8)
    with open(path, "wb") as f:
        f.write(struct.pack("<Q", len(text)))
        f.write(text)
        for b in blobs:
            f.write(b)


def read_model(folder):
    """(configuration, weights as float64) of a folder with config.json and one model.safetensors."""
    with open(os.path.join(folder, "config.json")) as f:
        cfg = json.load(f)
    with open(os.path.join(folder, "model.safetensors"), "rb") as f:
        (n,) = struct.unpack("<Q", f.read(8))
        header = json.loads(f.read(n))
        data = f.read()
    w = {}
    for name, info in header.items():
        if name == "__metadata__":
            continue
        blob = data[info["data_offsets"][0]:info["data_offsets"][1]]
        if info["dtype"] == "BF16":
            a = (np.frombuffer(blob, dtype=np.uint16).astype(np.uint32) << 16).view(np.float32)
        elif info["dtype"] == "F32":
            a = np.frombuffer(blob, dtype=np.float32)
        else:
            raise ValueError(f"{name}: dtype {info['dtype']}")
        w[name] = a.reshape(info["shape"]).astype(np.float64)
    return cfg, w


def write_model(folder, cfg, w, dtype="bfloat16"):
    os.makedirs(folder, exist_ok=True)
    with open(os.path.join(folder, "config.json"), "w") as f:
        json.dump(cfg, f)
    write_safetensors(os.path.join(folder, "model.safetensors"), w, dtype)
