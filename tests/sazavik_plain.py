"""A plain, slow Sazavik: whole sequences, no cache, float64, one function per mechanism.

It shares no code with the package; it reads the design's own configuration keys and the stored tensor names.
``forward(config, tensors, tokens)`` returns the logits [tokens, vocab]; ``streams``: a list that receives the residual
stream behind every layer; ``margins``: a list that receives, for every mixture of experts, how clear each token's
choice is.
"""
from __future__ import annotations

import math

import torch

from rounded_activations import activations_rounded, rnd

F64 = torch.float64


def rms_unit(x, eps):
    """x divided by its root mean square over the last dimension, eps inside the root."""
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)


def norm_around_one(x, weight, eps):
    """The norm of the stream and of the branches: its weight is stored as the distance from one."""
    return rms_unit(x, eps) * (1.0 + weight)


def rotate(x, positions, base, dims, neighbours):
    """x [T, heads, width]: pairs of the first ``dims`` dimensions turned by position * base^(-2i / dims); a pair is two
    neighbours (2i, 2i + 1) or (i, i + dims / 2)."""
    out = x.clone()
    for i in range(dims // 2):
        a, b = (2 * i, 2 * i + 1) if neighbours else (i, i + dims // 2)
        angle = positions.to(F64) * base ** (-2.0 * i / dims)
        cos, sin = torch.cos(angle)[:, None], torch.sin(angle)[:, None]
        out[..., a] = x[..., a] * cos - x[..., b] * sin
        out[..., b] = x[..., b] * cos + x[..., a] * sin
    return out


def in_window(T, size):
    """[T, T]: query i (row) sees the ``size`` latest keys up to its own; None: every earlier one."""
    i, j = torch.arange(T)[:, None], torch.arange(T)[None, :]
    return (j <= i) if size is None else (j <= i) & (i - j < size)


def in_chunk(T, size):
    """[T, T]: query i sees the keys up to its own that lie in its chunk of ``size`` positions."""
    i, j = torch.arange(T)[:, None], torch.arange(T)[None, :]
    return (j <= i) if size is None else (j <= i) & (i // size == j // size)


def slopes(heads):
    """Head h loses 2^(-8 (h + 1) / heads) of its score for every position between query and key."""
    return torch.tensor([2.0 ** (-8.0 * (h + 1) / heads) for h in range(heads)], dtype=F64)


def temperature(positions, coef, every):
    """What a query at position p is multiplied by: 1 + coef ln(floor((p + 1) / every) + 1)."""
    return 1.0 + coef * torch.log(torch.floor((positions.to(F64) + 1.0) / every) + 1.0)


def weighted_values(scores, seen, values, sinks=None):
    """scores [H, T, T], values [T, H, dv]: softmax over the seen keys; ``sinks`` [H]: one more term exp(sink) in a
    head's denominator, with no key and no value."""
    scores = scores.masked_fill(~seen[None], float("-inf"))
    top = scores.amax(dim=-1, keepdim=True)
    if sinks is not None:
        top = torch.maximum(top, sinks[:, None, None])
    e = torch.exp(scores - top)
    denominator = e.sum(dim=-1, keepdim=True)
    if sinks is not None:
        denominator = denominator + torch.exp(sinks[:, None, None] - top)
    return torch.einsum("hts,shd->thd", e / denominator, values)


# what tells the three attentions apart
FORMS = {
    "attention": dict(rotation="neighbours", mask=in_chunk, sink=True, gate=True, bias=False, distance=False, temperature=False),
    "attention_2": dict(rotation="halves", mask=in_chunk, sink=False, gate=False, bias=False, distance=False, temperature=False),
    "attention_3": dict(rotation=None, mask=in_window, sink=False, gate=True, bias=True, distance=True, temperature=True),
}


def head_norm(x, heads, weight, eps):
    """x [T, heads * dim]: every head over its root mean square, times a weight that all heads share."""
    return rms_unit(x.view(x.shape[0], heads, -1), eps) * weight


def keys_and_values(h, mixer, form, get, eps):
    """What a layer keeps of its tokens: normed (and turned) keys [T, G, dim] and values [T, G, vdim]."""
    T, G = h.shape[0], mixer["kv_heads"]
    k, v = h @ get("k").T, h @ get("v").T
    if form["bias"]:
        k, v = k + get("k.b"), v + get("v.b")
    k = head_norm(rnd(k), G, get("k.norm"), eps)
    if form["rotation"]:
        k = rotate(k, torch.arange(T), mixer["rot"]["base"], mixer["rot"]["dims"], form["rotation"] == "neighbours")
    return rnd(k), rnd(v).view(T, G, mixer["vdim"])


def attention(h, kind, mixer, get, eps, kept):
    """One mixer; ``get(name)``: its tensors; ``kept``: (keys, values) of this layer, or of the one it reads from."""
    form = FORMS[kind]
    T, H, G = h.shape[0], mixer["heads"], mixer["kv_heads"]
    positions = torch.arange(T)
    q = h @ get("q").T
    if form["bias"]:
        q = q + get("q.b")
    q = head_norm(rnd(q), H, get("q.norm"), eps)
    if form["rotation"]:
        q = rotate(q, positions, mixer["rot"]["base"], mixer["rot"]["dims"], form["rotation"] == "neighbours")
    if form["temperature"] and mixer.get("q_temp"):
        q = q * temperature(positions, mixer["q_temp"]["coef"], mixer["q_temp"]["every"])[:, None, None]
    k, v = (one.repeat_interleave(H // G, dim=1) for one in kept)
    scores = torch.einsum("thd,shd->hts", rnd(q), k) * mixer["scale"]
    if form["distance"]:
        away = (positions[:, None] - positions[None, :]).to(F64)
        scores = scores - slopes(H)[:, None, None] * away
    seen = form["mask"](T, (mixer.get("mask") or {}).get("size"))
    out = weighted_values(scores, seen, v, get("sink") if form["sink"] else None).reshape(T, -1)
    if form["gate"]:
        out = out * torch.sigmoid(rnd(h @ get("g").T))
    out = rnd(out) @ get("o").T
    if form["bias"]:
        out = out + get("o.b")
    return rnd(out)


def silu(z):
    return z * torch.sigmoid(z)


def clamped_feed_forward(h, get, limit):
    g = torch.clamp(rnd(h @ get("gate").T), max=limit)
    u = torch.clamp(rnd(h @ get("up").T), min=-limit, max=limit)
    return rnd(rnd(g * torch.sigmoid(1.702 * g) * (u + 1.0)) @ get("down").T)


def expert(h, get):
    return rnd(silu(h @ get("gate").T) * (h @ get("up").T)) @ get("down").T


def route(h, get, router):
    """(chosen [T, top], their scores [T, top], margin [T] of the choice): scores are sigmoids, not renormalized."""
    scores = torch.sigmoid(h @ get("router").T)
    ranked, order = torch.sort(scores, dim=-1, descending=True, stable=True)
    top = router["top"]
    margin = torch.full((h.shape[0],), float("inf"), dtype=F64)
    if top < scores.shape[1]:
        margin = ranked[:, top - 1] - ranked[:, top]
    return order[:, :top], ranked[:, :top], margin


def mixture(h, get, mlp, margins=None):
    """An expert is given its input times the token's weight for it; the outputs are added as they are."""
    chosen, weights, margin = route(h, get, mlp["router"])
    if margins is not None:
        margins.append(margin)
    out = torch.zeros_like(h)
    for number in range(mlp["router"]["experts"]):
        rows, places = torch.nonzero(chosen == number, as_tuple=True)
        if rows.numel():
            out[rows] += expert(weights[rows, places].reshape(-1, 1) * h[rows], lambda name: get(f"e{number}.{name}"))
    if mlp.get("shared") is not None:
        shared = rnd(expert(h, lambda name: get(f"shared.{name}")))
        out = out + torch.sigmoid(h @ get("shared.sg").T) * shared
    return out


def forward(config, tensors, tokens, streams=None, margins=None):
    eps = float(config["norm"]["eps"])
    whole = lambda name: tensors[name].to(F64)
    x = norm_around_one(whole("embed")[torch.as_tensor(tokens, dtype=torch.long)], whole("embed.norm"), eps)
    kept = {}
    for index, layer in enumerate(config["layers"]):
        of_layer = lambda name: whole(f"l{index}.{name}")
        of_mixer = lambda name: whole(f"l{index}.mix.{name}")
        mixer = layer["mixer"]
        h = rnd(norm_around_one(x, of_layer("norm1"), eps))
        source = mixer.get("kv_from")
        if source is None:
            source = index
            kept[index] = keys_and_values(h, mixer, FORMS[layer["type"]], of_mixer, eps)
        x = x + norm_around_one(attention(h, layer["type"], mixer, of_mixer, eps, kept[source]), of_layer("norm1b"), eps)
        mlp = layer.get("mlp")
        if mlp is not None:
            h = rnd(norm_around_one(x, of_layer("norm2"), eps))
            of_mlp = lambda name: whole(f"l{index}.mlp.{name}")
            if mlp["kind"] == "dense":
                branch = clamped_feed_forward(h, of_mlp, float(mlp["limit"]))
            else:
                branch = mixture(h, of_mlp, mlp, margins)
            x = x + norm_around_one(branch, of_layer("norm2b"), eps)
        if streams is not None:
            streams.append(x.clone())
    logits = rnd(norm_around_one(x, whole("final.norm"), eps)) @ whole("head").T
    cap = config.get("logit_softcap")
    return logits if cap is None else cap * torch.tanh(logits / cap)


def choice_margins(config, tensors, tokens):
    """Per position, by how much its closest choice of experts, in any layer, is decided."""
    margins = []
    forward(config, tensors, tokens, margins=margins)
    return torch.stack(margins).amin(dim=0) if margins else torch.full((len(tokens),), float("inf"), dtype=F64)


def rounding_noise(config, tensors, tokens, samples=6):
    """Per position, the largest departure of the logits that rounding the activations to 16 bits alone causes."""
    exact = forward(config, tensors, tokens)
    generator = torch.Generator().manual_seed(1)
    worst = torch.zeros(len(tokens), dtype=F64)
    for sample in range(samples):
        with activations_rounded(generator if sample else None):
            worst = torch.maximum(worst, (forward(config, tensors, tokens) - exact).abs().amax(dim=-1))
    return worst
