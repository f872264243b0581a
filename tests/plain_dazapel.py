"""A plain, slow implementation of the Dazapel decoder used only as the oracle of the tests.

Whole sequences from position 0, no cache, one function per mechanism, float64 arithmetic on
the CPU.  Nothing here imports the product package.  A model is a dictionary `cfg` (the
content of its config.json) and a dictionary of tensors under their checkpoint names.

Notation: T tokens, W the model's width; matrices are stored [out, in].
"""
from __future__ import annotations

import math

import torch

F64 = torch.float64
SWISH_ALPHA = 1.702


def f64(t):
    return t.to(F64)


def linear(x, weight, bias=None):
    y = f64(x) @ f64(weight).T
    return y if bias is None else y + f64(bias)


def sigmoid(x):
    return 1.0 / (1.0 + torch.exp(-x))


# ---------------------------------------------------------------------------- norms
def unit_rms(x, eps):
    """x / sqrt(mean(x^2) + eps) over the last axis."""
    x = f64(x)
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)


def rms_norm(x, weight, eps):
    return unit_rms(x, eps) * f64(weight)


# ---------------------------------------------------------------------------- rotation
def frequencies(rot):
    """f_i = base^(-2i / dims) for i < dims / 2; with a scaling, pairs that turn often within
    the original length keep their frequency, pairs that turn seldom are slowed by `factor`,
    and a linear ramp over i lies between."""
    dims, base = int(rot["dims"]), float(rot["base"])
    f = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
    scaling = rot.get("scaling")
    if not scaling:
        return f

    def index_of(turns):        # the pair that makes `turns` turns within the original length
        return dims * math.log(float(scaling["original"]) / (2.0 * math.pi * turns)) \
            / (2.0 * math.log(base))
    low = max(math.floor(index_of(float(scaling["fast"]))), 0)
    high = min(math.ceil(index_of(float(scaling["slow"]))), dims - 1)
    out = []
    for i, value in enumerate(f):
        ramp = min(max((i - low) / max(high - low, 0.001), 0.0), 1.0)
        out.append(value / float(scaling["factor"]) * ramp + value * (1.0 - ramp))
    return out


def magnitude(rot):
    """What cosine and sine are multiplied by."""
    scaling = rot.get("scaling")
    return 1.0 if not scaling else 0.1 * math.log(float(scaling["factor"])) + 1.0


def rotate_halves(x, positions, rot):
    """x [T, heads, dim]: the pairs (i, i + dims / 2) of the first dims elements of every head
    turn by position * f_i, scaled by the magnitude; the rest pass."""
    if not rot:
        return x
    half = int(rot["dims"]) // 2
    scale = magnitude(rot)
    out = x.clone()
    for i, f in enumerate(frequencies(rot)):
        angle = f64(positions) * f
        cos, sin = (torch.cos(angle) * scale)[:, None], (torch.sin(angle) * scale)[:, None]
        u, v = x[..., i], x[..., i + half]
        out[..., i] = u * cos - v * sin
        out[..., i + half] = v * cos + u * sin
    return out


# ---------------------------------------------------------------------------- attention
def visible_keys(i, mask):
    """The positions that position i sees: itself and what lies less than `size` back, and the
    sequence's first `keep_first` tokens however far back they lie."""
    if not mask or mask.get("size") is None:
        return list(range(i + 1))
    size, keep = int(mask["size"]), int(mask.get("keep_first") or 0)
    return [j for j in range(i + 1) if i - j < size or j < keep]


def softmax_attention(q, k, v, scale, visible):
    """q [T, H, d], k [T, G, d], v [T, G, e]; head h reads kv head h // (H / G); `visible(i)`
    gives the positions that row i sees.  Returns [T, H, e]."""
    T, H, _ = q.shape
    G = k.shape[1]
    out = torch.zeros(T, H, v.shape[2], dtype=F64)
    for i in range(T):
        seen = torch.as_tensor(visible(i))
        ks = k[seen].repeat_interleave(H // G, dim=1)          # [S, H, d]
        vs = v[seen].repeat_interleave(H // G, dim=1)
        scores = (ks * q[i][None]).sum(-1) * scale             # [S, H]
        weights = torch.softmax(scores, dim=0)
        out[i] = (weights[:, :, None] * vs).sum(dim=0)
    return out


def attention_mixer(h, tensors, prefix, mixer, eps, positions):
    """Biased projections, rotated queries and keys brought to unit RMS after the rotation, a
    window that keeps the first tokens, and a sigmoid gate on every element of the heads."""
    H, G = int(mixer["heads"]), int(mixer["kv_heads"])
    d, e = int(mixer["dim"]), int(mixer["vdim"])
    T = h.shape[0]

    def project(name, heads, size):
        return linear(h, tensors[prefix + name], tensors[prefix + name + ".b"]).reshape(T, heads, size)
    rot = mixer.get("rot")
    q = unit_rms(rotate_halves(project("q", H, d), positions, rot), eps)
    k = unit_rms(rotate_halves(project("k", G, d), positions, rot), eps)
    v = project("v", G, e)
    out = softmax_attention(q, k, v, float(mixer["scale"]),
                            lambda i: visible_keys(i, mixer.get("mask"))).reshape(T, H * e)
    out = out * sigmoid(linear(h, tensors[prefix + "g"]))
    return linear(out, tensors[prefix + "o"], tensors[prefix + "o.b"])


# ---------------------------------------------------------------------------- feed-forward
def clamped_expert(h, tensors, prefix, limit):
    """down(g sigmoid(1.702 g) (u + 1)) with g = min(gate h, limit), u = clamp(up h, +-limit)."""
    g = torch.clamp(linear(h, tensors[prefix + "gate"]), max=limit)
    u = torch.clamp(linear(h, tensors[prefix + "up"]), min=-limit, max=limit)
    return linear(g * sigmoid(SWISH_ALPHA * g) * (u + 1.0), tensors[prefix + "down"])


def choose(scores, router):
    """One row's scores [E] -> the chosen experts, best first; of equal scores the lower index.
    Experts form groups of neighbours; a group scores the sum of its two largest scores and
    only the best `keep` groups take part."""
    experts = scores.shape[0]
    groups = router.get("groups") or {"count": 1, "keep": 1}
    count, keep = int(groups["count"]), int(groups["keep"])
    size = experts // count
    values = scores.tolist()
    group_score = [sum(sorted(values[g * size:(g + 1) * size], reverse=True)[:2])
                   for g in range(count)]
    kept = sorted(range(count), key=lambda g: (-group_score[g], g))[:keep]
    allowed = [e for e in range(experts) if e // size in kept]
    return sorted(allowed, key=lambda e: (-values[e], e))[:int(router["top"])]


def margin_of(scores, router):
    """How close one row's choice is to another one, in units of the score: the least of the
    gap between the last kept and the first dropped group's score, and the gap between the
    last chosen and the first unchosen score of the kept groups' experts."""
    experts = scores.shape[0]
    groups = router.get("groups") or {"count": 1, "keep": 1}
    count, keep, top = int(groups["count"]), int(groups["keep"]), int(router["top"])
    size = experts // count
    values = scores.tolist()
    group_score = [sum(sorted(values[g * size:(g + 1) * size], reverse=True)[:2])
                   for g in range(count)]
    order = sorted(range(count), key=lambda g: (-group_score[g], g))
    gap = float("inf")
    if keep < count:
        gap = group_score[order[keep - 1]] - group_score[order[keep]]
    ranked = sorted((values[e] for e in range(experts) if e // size in order[:keep]), reverse=True)
    if top < len(ranked):
        gap = min(gap, ranked[top - 1] - ranked[top])
    return gap


def route(h, tensors, prefix, router):
    """(chosen experts [T, top], their weights [T, top], scores [T, E])."""
    scores = sigmoid(linear(h, tensors[prefix + "router"]))
    chosen = torch.tensor([choose(row, router) for row in scores])
    picked = torch.gather(scores, 1, chosen)
    return chosen, picked / (picked.sum(-1, keepdim=True) + 1e-20) * float(router["scale"]), scores


def routed_feed_forward(h, tensors, prefix, mlp, margins=None):
    h = f64(h)
    chosen, weights, scores = route(h, tensors, prefix, mlp["router"])
    if margins is not None:
        margins.append(torch.tensor([margin_of(row, mlp["router"]) for row in scores]))
    limit = float(mlp["expert"]["limit"])
    out = torch.zeros_like(h)
    for e in sorted(set(chosen.flatten().tolist())):
        rows, places = (chosen == e).nonzero(as_tuple=True)
        out[rows] += weights[rows, places][:, None] * clamped_expert(h[rows], tensors,
                                                                     f"{prefix}e{e}.", limit)
    if mlp.get("shared"):
        out = out + clamped_expert(h, tensors, prefix + "shared.", float(mlp["shared"]["limit"]))
    return out


# ---------------------------------------------------------------------------- the model
def layer_runs(cfg):
    """(layer, number of the pass that this run begins or None) in the order of execution."""
    loop = cfg.get("loop")
    n = len(cfg["layers"])
    if not loop:
        return [(i, None) for i in range(n)]
    start, stop, times = int(loop["start"]), int(loop["stop"]), int(loop["times"])
    runs = [(i, None) for i in range(start)]
    for t in range(times):
        runs += [(i, t if i == start else None) for i in range(start, stop)]
    return runs + [(i, None) for i in range(stop, n)]


def forward(cfg, tensors, tokens, layer_outputs=None, margins=None):
    """Logits [T, vocab] of one sequence of token ids from position 0.  `layer_outputs`: a
    list that receives the stream after every run of a layer; `margins`: a list that receives,
    for every run of a routed feed-forward, the rows' choice margins."""
    eps, mult = float(cfg["norm"]["eps"]), float(cfg["residual_mult"])
    tokens = torch.as_tensor(tokens, dtype=torch.int64)
    positions = torch.arange(tokens.shape[0])
    x = f64(tensors["embed"])[tokens]
    for index, begins in layer_runs(cfg):
        layer, name = cfg["layers"][index], f"l{index}."
        if begins is not None:
            x = x + f64(tensors["loop.step"])[begins]
        if layer["type"] != "attention":
            raise ValueError(f"unknown layer type {layer['type']!r}")
        a = attention_mixer(rms_norm(x, tensors[name + "norm1"], eps), tensors, name + "mix.",
                            layer["mixer"], eps, positions)
        x = x + mult * rms_norm(a, tensors[name + "norm1b"], eps)
        if layer.get("mlp") is not None:
            f = routed_feed_forward(rms_norm(x, tensors[name + "norm2"], eps), tensors,
                                    name + "mlp.", layer["mlp"], margins)
            x = x + mult * rms_norm(f, tensors[name + "norm2b"], eps)
        if layer_outputs is not None:
            layer_outputs.append(x.clone())
    return linear(rms_norm(x, tensors["final.norm"], eps), tensors["embed"])


def clear_rows(cfg, tensors, tokens, margin, carry=True):
    """(logits, mask of the positions whose logits no routing decision closer than `margin`
    can have touched).  `carry`: a close call at a position also touches every later one (the
    caches carry it on)."""
    margins = []
    logits = forward(cfg, tensors, tokens, margins=margins)
    clear = torch.ones(logits.shape[0], dtype=torch.bool)
    for rows in margins:
        clear &= rows >= margin
    if carry and not bool(clear.all()):
        first = int((~clear).nonzero()[0])
        clear[first:] = False
    return logits, clear
