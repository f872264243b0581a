"""A plain, slow implementation of the Lemotar decoder used only as the oracle of the tests.

Whole sequences from position 0, no cache, token-by-token recurrences, keys and values of
latent attention expanded for every head, one function per mechanism, float64 arithmetic on
the CPU.  Nothing here imports the product package.  A model is a dictionary `cfg` (the
content of its config.json) and a dictionary of tensors under their checkpoint names.

Notation: T tokens, W the model's width; matrices are stored [out, in].
"""
from __future__ import annotations

import math

import torch

F64 = torch.float64


def f64(t):
    return t.to(F64)


def linear(x, weight):
    return f64(x) @ f64(weight).T


def sigmoid(x):
    return 1.0 / (1.0 + torch.exp(-x))


def silu(x):
    return x * sigmoid(x)


def softplus(x):
    return torch.clamp(x, min=0.0) + torch.log1p(torch.exp(-x.abs()))


# ---------------------------------------------------------------------------- norms
def unit_rms(x, eps):
    """x / sqrt(mean(x^2) + eps) over the last axis."""
    x = f64(x)
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)


def rms_norm(x, weight, eps):
    return unit_rms(x, eps) * f64(weight)


def offset_norm(x, weight, eps):
    """An RMS norm whose stored weight is its distance from one."""
    return unit_rms(x, eps) * (1.0 + f64(weight))


# ---------------------------------------------------------------------------- rotation
def plain_frequencies(base, dims):
    return [float(base) ** (-2.0 * i / dims) for i in range(dims // 2)]


def stretched_frequencies(rot):
    """(frequencies, what cosine and sine are multiplied by): with `scaling`, pairs that turn
    more than `fast` times within the original length keep their frequency, pairs that turn
    less than `slow` times have it divided by the factor, linear in the pair's index between."""
    base, dims = float(rot["base"]), int(rot["dims"])
    freqs = plain_frequencies(base, dims)
    s = rot.get("scaling")
    if not s:
        return freqs, 1.0
    factor = float(s["factor"])

    def pair_of(turns):
        return dims * math.log(float(s["original"]) / (2.0 * math.pi * turns)) / (2.0 * math.log(base))
    first = max(math.floor(pair_of(float(s["fast"]))), 0)
    last = min(math.ceil(pair_of(float(s["slow"]))), dims - 1)
    out = []
    for i, f in enumerate(freqs):
        share = min(1.0, max(0.0, (i - first) / max(last - first, 0.001)))
        out.append(f / factor * share + f * (1.0 - share))
    return out, 0.1 * math.log(factor) + 1.0


def rotate_neighbours(x, positions, rot):
    """x [T, heads, dim]: elements (2i, 2i + 1), i < dims / 2, of every head turn by
    position * f_i; the rest pass."""
    out = x.clone()
    freqs, magnitude = stretched_frequencies(rot)
    for i, f in enumerate(freqs):
        angle = f64(positions) * f
        cos, sin = (magnitude * torch.cos(angle))[:, None], (magnitude * torch.sin(angle))[:, None]
        u, v = x[..., 2 * i], x[..., 2 * i + 1]
        out[..., 2 * i] = u * cos - v * sin
        out[..., 2 * i + 1] = v * cos + u * sin
    return out


def rotate_halves(x, positions, rot):
    """The same for the pairs (i, i + dims / 2)."""
    out = x.clone()
    freqs, magnitude = stretched_frequencies(rot)
    half = len(freqs)
    for i, f in enumerate(freqs):
        angle = f64(positions) * f
        cos, sin = (magnitude * torch.cos(angle))[:, None], (magnitude * torch.sin(angle))[:, None]
        u, v = x[..., i], x[..., i + half]
        out[..., i] = u * cos - v * sin
        out[..., i + half] = v * cos + u * sin
    return out


# ---------------------------------------------------------------------------- attention
def window_attention(q, k, v, scale, window, sink, softcap=None):
    """q [T, H, d], k [T, G, d], v [T, G, e]; head h reads kv head h // (H / G); query i sees the
    keys j with 0 <= i - j < window (None: all j <= i).  Scores are scaled, then capped
    c tanh(s / c); the softmax's denominator also holds exp(sink[h]).  Returns [T, H, e]."""
    T, H, _ = q.shape
    G = k.shape[1]
    out = torch.zeros(T, H, v.shape[2], dtype=F64)
    for i in range(T):
        lo = 0 if window is None else max(0, i - window + 1)
        for g in range(G):
            heads = slice(g * (H // G), (g + 1) * (H // G))
            scores = (q[i, heads] @ k[lo:i + 1, g].T) * scale            # [H / G, keys]
            if softcap is not None:
                scores = softcap * torch.tanh(scores / softcap)
            extra = sink[heads][:, None]
            top = torch.maximum(scores.max(dim=1, keepdim=True).values, extra)
            e = torch.exp(scores - top)
            weights = e / (e.sum(dim=1, keepdim=True) + torch.exp(extra - top))
            out[i, heads] = weights @ v[lo:i + 1, g]
    return out


def shared_value_attention(h, tensors, prefix, mixer, eps, positions):
    """The softmax half of the parallel mixer: values are the keys as projected, queries and
    keys normed over the whole projection and then rotated, capped scores, a window, a one in
    the softmax's denominator."""
    H, G, d = int(mixer["heads"]), int(mixer["kv_heads"]), int(mixer["dim"])
    T = h.shape[0]
    q, k = linear(h, tensors[prefix + "q"]), linear(h, tensors[prefix + "k"])
    v = k.reshape(T, G, d)
    q = rms_norm(q, tensors[prefix + "q.norm"], eps).reshape(T, H, d)
    k = rms_norm(k, tensors[prefix + "k.norm"], eps).reshape(T, G, d)
    q, k = rotate_neighbours(q, positions, mixer["rot"]), rotate_neighbours(k, positions, mixer["rot"])
    mask = mixer.get("mask")
    out = window_attention(q, k, v, float(mixer["scale"]), int(mask["size"]) if mask else None,
                           torch.zeros(H, dtype=F64), float(mixer["softcap"]))
    return linear(out.reshape(T, H * d), tensors[prefix + "o"])


def latent_attention(h, tensors, prefix, mixer, eps, positions, shared):
    """Per position a normed latent and one rotated key part shared by the heads; unrotated keys
    and values are up-projections of the latent.  `shared`: (latent, rotated part) of the layer
    whose cache this layer reads, or None.  Returns (output [T, W], (latent, rotated part))."""
    H, d, r = int(mixer["heads"]), int(mixer["dim"]), int(mixer["rot_dim"])
    e, rank = int(mixer["vdim"]), int(mixer["kv_rank"])
    T = h.shape[0]
    q = linear(h, tensors[prefix + "q"]).reshape(T, H, d + r)
    turned = rotate_halves(q[..., d:], positions, mixer["rot"])
    if shared is None:
        down = linear(h, tensors[prefix + "dkv"])
        latent = rms_norm(down[:, :rank], tensors[prefix + "dkv.norm"], eps)
        part = rotate_halves(down[:, None, rank:], positions, mixer["rot"])[:, 0]
    else:
        latent, part = shared
    k_plain = linear(latent, tensors[prefix + "uk"]).reshape(T, H, d)
    v = linear(latent, tensors[prefix + "uv"]).reshape(T, H, e)
    k = torch.cat([k_plain, part[:, None, :].expand(T, H, r)], dim=2)
    mask = mixer.get("mask")
    out = window_attention(torch.cat([q[..., :d], turned], dim=2), k, v, float(mixer["scale"]),
                           int(mask["size"]) if mask else None, f64(tensors[prefix + "sink"]))
    out = out.reshape(T, H * e) * sigmoid(linear(h, tensors[prefix + "g"]))
    return linear(out, tensors[prefix + "o"]), (latent, part)


# ---------------------------------------------------------------------------- gated delta rule
def short_convolution(x, taps_weight):
    """x [T, C], taps_weight [C, taps]: y_t = sum_j w[:, j] x_(t - taps + 1 + j), inputs before
    the sequence's start being zero; then silu."""
    x, w = f64(x), f64(taps_weight)
    taps = w.shape[1]
    out = torch.zeros_like(x)
    for t in range(x.shape[0]):
        for j in range(taps):
            s = t - taps + 1 + j
            if s >= 0:
                out[t] += w[:, j] * x[s]
    return silu(out)


def unit_vector(x):
    return x / torch.sqrt((x * x).sum(dim=-1, keepdim=True) + 1e-6)


def delta_recurrence(q, k, v, beta, decay):
    """q, k [T, H, d] (one per head already), v [T, H, e], beta [T, H], decay [T, H, d]: per head
    S <- diag(decay) S; u = beta (v - S^T k); S <- S + k u^T; o = S^T q.  Returns [T, H, e]."""
    T, H, d = q.shape
    state = torch.zeros(H, d, v.shape[2], dtype=F64)
    out = torch.zeros(T, H, v.shape[2], dtype=F64)
    for t in range(T):
        state = state * decay[t][:, :, None]
        seen = (state * k[t][:, :, None]).sum(dim=1)
        u = beta[t][:, None] * (v[t] - seen)
        state = state + k[t][:, :, None] * u[:, None, :]
        out[t] = (state * q[t][:, :, None]).sum(dim=1)
    return out


def channel_decay(h, tensors, prefix, heads, dim):
    """g [T, heads, dim] = exp(-exp(A_log_h) softplus(W_a2 (W_a1 h) + dt_bias))."""
    z = linear(linear(h, tensors[prefix + "a1"]), tensors[prefix + "a2"]) + f64(tensors[prefix + "dt_bias"])
    rate = torch.exp(f64(tensors[prefix + "A_log"]))
    return torch.exp(-rate[None, :, None] * softplus(z).reshape(h.shape[0], heads, dim))


def delta_mixer(h, tensors, prefix, mixer, eps):
    H, G = int(mixer["heads"]), int(mixer["kv_heads"])
    d, e = int(mixer["dim"]), int(mixer["vdim"])
    T = h.shape[0]

    def convolved(name, heads, size):
        x = short_convolution(linear(h, tensors[prefix + name]), tensors[prefix + name + ".conv"])
        return x.reshape(T, heads, size)
    q = unit_vector(convolved("q", G, d)) * d ** -0.5
    k = unit_vector(convolved("k", G, d))
    v = convolved("v", H, e)
    shared = torch.arange(H) // (H // G)
    beta = sigmoid(linear(h, tensors[prefix + "b"]))
    decay = channel_decay(h, tensors, prefix, H, d)
    o = delta_recurrence(q[:, shared], k[:, shared], v, beta, decay)
    o = rms_norm(o, tensors[prefix + "norm"], eps).reshape(T, H * e)
    o = o * sigmoid(linear(linear(h, tensors[prefix + "g1"]), tensors[prefix + "g2"]))
    return linear(o, tensors[prefix + "o"])


def parallel_mixer(h, tensors, prefix, mixer, eps, positions):
    """Half the sum of the two mixers' outputs, each RMS-normed over the width first."""
    left = shared_value_attention(h, tensors, prefix + "left.", mixer["left"], eps, positions)
    right = delta_mixer(h, tensors, prefix + "right.", mixer["right"], eps)
    return 0.5 * (rms_norm(left, tensors[prefix + "left.out"], eps)
                  + rms_norm(right, tensors[prefix + "right.out"], eps))


# ---------------------------------------------------------------------------- the rest
def dense_feed_forward(h, tensors, prefix):
    return linear(silu(linear(h, tensors[prefix + "gate"])) * linear(h, tensors[prefix + "up"]),
                  tensors[prefix + "down"])


def forward(cfg, tensors, tokens, layer_outputs=None):
    """Logits [T, vocab] of one sequence of token ids from position 0.  `layer_outputs`: a
    list that receives the stream after every layer."""
    eps = float(cfg["norm"]["eps"])
    alpha = float(cfg["postln_alpha"])
    tokens = torch.as_tensor(tokens, dtype=torch.int64)
    positions = torch.arange(tokens.shape[0])
    x = f64(tensors["embed"])[tokens] * float(cfg["embedding"]["scale"])
    kept = {}
    for index, layer in enumerate(cfg["layers"]):
        name, mixer = f"l{index}.", layer["mixer"]
        if layer["type"] == "parallel":
            a = parallel_mixer(x, tensors, name + "mix.", mixer, eps, positions)
        elif layer["type"] == "latent_attention":
            source = mixer.get("kv_from")
            a, kept[index] = latent_attention(x, tensors, name + "mix.", mixer, eps, positions,
                                              None if source is None else kept[int(source)])
        else:
            raise ValueError(f"unknown layer type {layer['type']!r}")
        x = offset_norm(alpha * x + a, tensors[name + "norm1"], eps)
        if layer.get("mlp") is not None:
            f = dense_feed_forward(x, tensors, name + "mlp.")
            x = offset_norm(alpha * x + f, tensors[name + "norm2"], eps)
        if layer_outputs is not None:
            layer_outputs.append(x.clone())
    x = offset_norm(x, tensors["final.norm"], eps)
    return linear(x, tensors["head"])
