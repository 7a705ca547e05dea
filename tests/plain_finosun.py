"""A plain, slow implementation of the Finosun design in NumPy float64, one function per
mechanism, written from the design's equations.  It shares no code with the library: the
tests hold the engine against it.

Notation: a sequence's tokens are rows; positions count from 0.  `cfg` is the model's
configuration as a dict (the keys of its config.json), `w` maps tensor names to float arrays.
A layer is x += s1 * mixer(norm1(x)), x += s2 * feed_forward(norm2(x)), s1 and s2 learnt
vectors of the model's width.
"""
from __future__ import annotations

import json
import math
import os
import struct

import numpy as np

ALPHA = 1.702


# ------------------------------------------------------------------ mechanisms ------
def rms_divide(x, eps):
    """x / sqrt(mean(x^2) + eps) over the last axis."""
    return x / np.sqrt((x * x).mean(axis=-1, keepdims=True) + eps)


def rms_norm(x, weight, eps):
    return rms_divide(x, eps) * weight


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def softmax(z):
    p = np.exp(z - z.max(axis=-1, keepdims=True))
    return p / p.sum(axis=-1, keepdims=True)


def turn(x, positions, dims, base, neighbours):
    """x [T, heads, d]: the first `dims` elements of every head in pairs, element 2i with 2i + 1 (`neighbours`) or i
    with i + dims/2; pair i is turned by position * base^(-2i/dims), the elements behind pass."""
    y = np.array(x, dtype=np.float64)
    for i in range(dims // 2):
        a, b = (2 * i, 2 * i + 1) if neighbours else (i, i + dims // 2)
        ang = np.asarray(positions, dtype=np.float64)[:, None] * base ** (-2.0 * i / dims)
        y[..., a] = x[..., a] * np.cos(ang) - x[..., b] * np.sin(ang)
        y[..., b] = x[..., b] * np.cos(ang) + x[..., a] * np.sin(ang)
    return y


def causal(T):
    return np.tril(np.ones((T, T), dtype=bool))


def window(T, size):
    """Key j is seen by query i when 0 <= i - j < size."""
    i = np.arange(T)
    return causal(T) & ((i[:, None] - i[None, :]) < size)


def softmax_attention(q, k, v, scales, visible):
    """q [T, H, d], k [T, G, d], v [T, G, e] -> [T, H, e]; query head h reads key/value head h // (H / G), its scores
    are (q . k) scales[h]; visible [T, T] (row: query, column: key)."""
    T, H, _ = q.shape
    G = k.shape[1]
    out = np.zeros((T, H, v.shape[2]))
    for h in range(H):
        g = h // (H // G)
        s = np.where(visible, (q[:, h] @ k[:, g].T) * scales[h], -np.inf)
        out[:, h] = softmax(s) @ v[:, g]
    return out


def clamped_unit(h, gate, up, down, limit):
    """g sigmoid(1.702 g) (u + 1) through `down`, g bounded from above and u on both sides."""
    g = np.minimum(h @ gate.T, limit)
    u = np.clip(h @ up.T, -limit, limit)
    return (g * sigmoid(ALPHA * g) * (u + 1.0)) @ down.T


def choose_outputs(z, correction, top):
    """z [T, N] router logits (experts, then identities).  s = softmax(z); the `top` largest s + correction are
    chosen (ties to the lower number), their weights are s as it is.  -> (chosen [T, top], weights [T, top])."""
    s = softmax(z)
    chosen = np.argsort(-(s + correction[None, :]), axis=1, kind="stable")[:, :top]
    return chosen, np.take_along_axis(s, chosen, axis=1)


def join_input(x, x0, w_in):
    """W_in applied to the residual rows and the embedding output side by side."""
    return np.concatenate([x, x0], axis=1) @ w_in.T


# ------------------------------------------------------------------ mixers ----------
def attention_mixer(h, w, p, m, eps, positions):
    """Grouped heads in a sliding window: one norm over the whole query (key) projection, part of every head rotated
    in pairs of neighbours, every head's value divided by its root mean square, a learnt factor on a head's scores."""
    T = h.shape[0]
    H, G, d, e = m["heads"], m.get("kv_heads", m["heads"]), m["dim"], m.get("vdim", m["dim"])
    q = rms_norm(h @ w[p + "q"].T, w[p + "q.norm"], eps).reshape(T, H, d)
    k = rms_norm(h @ w[p + "k"].T, w[p + "k.norm"], eps).reshape(T, G, d)
    v = rms_divide((h @ w[p + "v"].T).reshape(T, G, e), eps)
    rot = m.get("rot")
    if rot:
        q = turn(q, positions, rot["dims"], rot["base"], True)
        k = turn(k, positions, rot["dims"], rot["base"], True)
    size = (m.get("mask") or {}).get("size")
    visible = window(T, size) if size else causal(T)
    o = softmax_attention(q, k, v, m["scale"] * w[p + "temp"], visible)
    return o.reshape(T, H * e) @ w[p + "o"].T


def latent_mixer(h, w, p, m, eps, positions):
    """Keys and values of every head from one normed latent a token, beside one rotated key part all heads share; the
    heads' outputs pass a sigmoid gate element by element."""
    T = h.shape[0]
    H, d, r, e, rank = m["heads"], m["dim"], m["rot_dim"], m.get("vdim", m["dim"]), m["kv_rank"]
    q = (h @ w[p + "q"].T).reshape(T, H, d + r)
    low = h @ w[p + "dkv"].T
    c = rms_norm(low[:, :rank], w[p + "dkv.norm"], eps)
    k_rot = low[:, rank:].reshape(T, 1, r)
    rot = m.get("rot")
    q_rot = q[..., d:]
    if r and rot:
        q_rot = turn(q_rot, positions, rot["dims"], rot["base"], False)
        k_rot = turn(k_rot, positions, rot["dims"], rot["base"], False)
    q = np.concatenate([q[..., :d], q_rot], axis=2)
    k = np.concatenate([(c @ w[p + "uk"].T).reshape(T, H, d), np.repeat(k_rot, H, axis=1)], axis=2)
    v = (c @ w[p + "uv"].T).reshape(T, H, e)
    o = softmax_attention(q, k, v, np.full(H, m["scale"]), causal(T)).reshape(T, H * e)
    return (o * sigmoid(h @ w[p + "g"].T)) @ w[p + "o"].T


MIXERS = {"attention": attention_mixer, "latent_attention": latent_mixer}


# ------------------------------------------------------------------ feed-forward ----
def feed_forward(h, w, p, f):
    r = f["router"]
    chosen, weights = choose_outputs(h @ w[p + "router"].T, w[p + "correction"], r["top"])
    out = np.zeros_like(h)
    for t in range(h.shape[0]):
        for j, share in zip(chosen[t], weights[t]):
            if j >= r["experts"]:
                out[t] += share * h[t]
            else:
                q = p + "e%d." % j
                out[t] += share * clamped_unit(h[t:t + 1], w[q + "gate"], w[q + "up"], w[q + "down"], f["expert"]["limit"])[0]
    if f.get("shared"):
        q = p + "shared."
        out += sigmoid(h @ w[q + "sg"].T) * clamped_unit(h, w[q + "gate"], w[q + "up"], w[q + "down"], f["shared"]["limit"])
    return out


# ------------------------------------------------------------------ the model -------
def layer_runs(cfg):
    """(layer, whether the embedding output is joined in right before it), in the order of running."""
    n = len(cfg["layers"])
    loop = cfg.get("loop")
    if not loop:
        return [(i, False) for i in range(n)]
    a, b, times = loop["start"], loop["stop"], loop.get("times", 1)
    return ([(i, False) for i in range(a)] + [(i, i == a) for _ in range(times) for i in range(a, b)]
            + [(i, False) for i in range(b, n)])


def forward(cfg, w, tokens, return_layers=False):
    """Logits [T, vocab] of one sequence from position 0 (and the residual rows after every layer run)."""
    eps = cfg["norm"]["eps"]
    x0 = x = w["embed"][np.asarray(tokens)]
    positions = np.arange(len(tokens))
    rows = []
    for i, joined in layer_runs(cfg):
        if joined:
            x = join_input(x, x0, w["loop.in"])
        layer, p = cfg["layers"][i], "l%d." % i
        h = rms_norm(x, w[p + "norm1"], eps)
        x = x + w[p + "ls1"] * MIXERS[layer["type"]](h, w, p + "mix.", layer["mixer"], eps, positions)
        if layer.get("mlp"):
            x = x + w[p + "ls2"] * feed_forward(rms_norm(x, w[p + "norm2"], eps), w, p + "mlp.", layer["mlp"])
        rows.append(x)
    logits = rms_norm(x, w["final.norm"], eps) @ w["embed"].T
    return (logits, np.stack(rows)) if return_layers else logits


def greedy(cfg, w, prompt, n):
    tokens = list(prompt)
    for _ in range(n):
        tokens.append(int(np.argmax(forward(cfg, w, tokens)[-1])))
    return tokens[len(prompt):]


# ------------------------------------------------------------------ weights ---------
def tensor_shapes(cfg):
    """name -> shape of every tensor of a model of this configuration."""
    W, V = cfg["width"], cfg["vocab"]
    out = {"embed": (V, W)}
    if cfg.get("loop"):
        out["loop.in"] = (W, 2 * W)
    for i, layer in enumerate(cfg["layers"]):
        p, m, f = "l%d." % i, layer["mixer"], layer.get("mlp")
        out[p + "norm1"] = out[p + "ls1"] = (W,)
        if f:
            out[p + "norm2"] = out[p + "ls2"] = (W,)
        q = p + "mix."
        if layer["type"] == "attention":
            H, G, d, e = m["heads"], m.get("kv_heads", m["heads"]), m["dim"], m.get("vdim", m["dim"])
            out[q + "q"], out[q + "k"], out[q + "v"] = (H * d, W), (G * d, W), (G * e, W)
            out[q + "q.norm"], out[q + "k.norm"], out[q + "temp"] = (H * d,), (G * d,), (H,)
            out[q + "o"] = (W, H * e)
        else:
            H, d, r, e, rank = m["heads"], m["dim"], m["rot_dim"], m.get("vdim", m["dim"]), m["kv_rank"]
            out[q + "q"], out[q + "dkv"], out[q + "dkv.norm"] = (H * (d + r), W), (rank + r, W), (rank,)
            out[q + "uk"], out[q + "uv"] = (H * d, rank), (H * e, rank)
            out[q + "g"], out[q + "o"] = (H * e, W), (W, H * e)
        if not f:
            continue
        q, r = p + "mlp.", f["router"]
        for j in range(r["experts"]):
            n = f["expert"]["ff"]
            out[q + "e%d.gate" % j], out[q + "e%d.up" % j], out[q + "e%d.down" % j] = (n, W), (n, W), (W, n)
        n = r["experts"] + r.get("identity", 0)
        out[q + "router"], out[q + "correction"] = (n, W), (n,)
        if f.get("shared"):
            n = f["shared"]["ff"]
            out[q + "shared.gate"], out[q + "shared.up"], out[q + "shared.down"] = (n, W), (n, W), (W, n)
            out[q + "shared.sg"] = (1, W)
    out["final.norm"] = (W,)
    return out


def to_bf16_values(a):
    """Round float64 values to the nearest bfloat16 (ties to even), returned as float64."""
    u = np.asarray(a, dtype=np.float32).view(np.uint32).astype(np.uint64)
    u = ((u + 0x7FFF + ((u >> 16) & 1)) >> 16) << 16
    return u.astype(np.uint32).view(np.float32).astype(np.float64)


def random_weights(cfg, seed, router_spread=0.0, gain=1.0):
    """Weights that keep every activation of order one, already rounded to bfloat16.  `router_spread` puts the
    outputs' corrections that far apart, so that a bfloat16 run chooses as the float64 run does; `gain` sizes the
    matrices."""
    rng = np.random.default_rng(seed)
    w = {}
    for name, shape in tensor_shapes(cfg).items():
        tail = name.split(".")[-1]
        if "norm" in tail:
            a = 1.0 + 0.2 * rng.standard_normal(shape)
        elif tail in ("ls1", "ls2"):
            a = 0.6 + 0.25 * rng.standard_normal(shape)
        elif tail == "temp":
            a = 1.0 + 0.4 * rng.standard_normal(shape)
        elif tail == "correction":
            a = 0.2 * rng.standard_normal(shape) + router_spread * rng.permutation(shape[0])
        elif name == "embed":
            a = rng.standard_normal(shape)
        elif name == "loop.in":
            a = rng.standard_normal(shape) * (0.9 / math.sqrt(shape[-1]))
        else:
            a = rng.standard_normal(shape) * (1.5 * gain / math.sqrt(shape[-1]))
        w[name] = to_bf16_values(a)
    return w


def write_safetensors(path, w, dtype="bfloat16"):
    """Write `w` as one safetensors file of bfloat16 (or float32) tensors."""
    header, blobs, at = {}, [], 0
    for name, a in w.items():
        a32 = np.ascontiguousarray(a, dtype=np.float32)
        if dtype == "bfloat16":
            blob = (a32.view(np.uint32) >> 16).astype(np.uint16).tobytes()
            tag = "BF16"
        else:
            blob, tag = a32.tobytes(), "F32"
        header[name] = {"dtype": tag, "shape": list(a32.shape), "data_offsets": [at, at + len(blob)]}
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
