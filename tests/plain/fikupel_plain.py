"""A plain, slow Fikupel: whole sequences, no cache, one function per mechanism.

It shares no code with the engine.  Every function works on one sequence, [tokens, ...] torch tensors on
the CPU, in the precision of the tensors it is given (float32, or float64 to see how much of a
difference is rounding).  Weights come as a dict from tensor name to tensor; `cfg` is config.json as a
dict.

Notation: T tokens, W the model's width, H query heads, G key heads, dk and dv a head's key and value
sizes, n the copies of the stream; `p(name)` is a layer's tensor.
"""
from __future__ import annotations

import math

import torch


# ----------------------------------------------------------------------------
# small pieces
# ----------------------------------------------------------------------------

def rms_norm(x, weight, eps):
    """y = x / sqrt(mean(x^2) + eps) [* weight], over the last dimension."""
    y = x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)
    return y if weight is None else y * weight


def silu(z):
    return z * torch.sigmoid(z)


def stretched_frequencies(dims, base, scaling):
    """The frequency of every pair i < dims / 2, f = base^(-2i/dims), in 64-bit.  With scaling (factor, low, high,
    original) a pair is judged by how many of its wavelengths 2 pi / f fit into `original`: more than `high`: it stays;
    fewer than `low`: it is slowed down by `factor`; between the two a blend that is linear in that number."""
    out = []
    for i in range(dims // 2):
        f = float(base) ** (-2.0 * i / dims)
        if scaling:
            factor, low, high = (float(scaling[k]) for k in ("factor", "low", "high"))
            waves = float(scaling["original"]) * f / (2.0 * math.pi)
            if waves < low:
                f = f / factor
            elif waves <= high:
                s = (waves - low) / (high - low)
                f = (1.0 - s) * f / factor + s * f
        out.append(f)
    return torch.tensor(out, dtype=torch.float64)


def turn_pairs(x, positions, freq, sign=1.0):
    """x [T, n, d]: entries 2i and 2i + 1 of each vector, for i < len(freq), are turned by the angle
    sign * position * freq[i]; the entries behind them stay."""
    out = x.clone()
    k = 2 * len(freq)
    if k:
        ang = sign * positions.to(torch.float64)[:, None] * freq[None, :]
        cos, sin = torch.cos(ang).to(x.dtype)[:, None, :], torch.sin(ang).to(x.dtype)[:, None, :]
        a, b = x[..., 0:k:2], x[..., 1:k:2]
        out[..., 0:k:2] = a * cos - b * sin
        out[..., 1:k:2] = b * cos + a * sin
    return out


def seen_keys(T, window, keep):
    """[T, T] (query, key): the query at i sees j <= i if j is one of the `window` last (i - j < window; None: all) or one
    of the first `keep`."""
    i = torch.arange(T)[:, None]
    j = torch.arange(T)[None, :]
    near = (i - j < window) if window else torch.ones(T, T, dtype=torch.bool)
    return (j <= i) & (near | (j < (keep or 0)))


def sink_softmax(scores, seen, sink):
    """scores [H, T, T]: exp(score) over the seen keys, divided by their sum and exp(sink[h])."""
    s = scores.masked_fill(~seen, float("-inf"))
    b = sink[:, None, None].to(s.dtype).expand(-1, s.shape[1], 1)
    return torch.softmax(torch.cat([s, b], dim=-1), dim=-1)[..., :-1]


# ----------------------------------------------------------------------------
# mixers
# ----------------------------------------------------------------------------

def attention(h, p, m, eps):
    """q and k normed per head, turned by the position; values turned by theirs over their whole width; scores times scale
    and a number per head; window and kept first tokens; sink; results turned back, gated entry by entry, projected."""
    T = h.shape[0]
    H, G, dk, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    pos = torch.arange(T)
    q = rms_norm((h @ p("q").T).view(T, H, dk), p("q.norm"), eps)
    k = rms_norm((h @ p("k").T).view(T, G, dk), p("k.norm"), eps)
    v = (h @ p("v").T).view(T, G, dv)
    rot = m["rot"]
    freq = stretched_frequencies(rot["dims"], rot["base"], rot.get("scaling"))
    vfreq = stretched_frequencies(dv, rot["base"], None)
    q, k, v = turn_pairs(q, pos, freq), turn_pairs(k, pos, freq), turn_pairs(v, pos, vfreq)
    k, v = k.repeat_interleave(H // G, dim=1), v.repeat_interleave(H // G, dim=1)
    scores = torch.einsum("ihd,jhd->hij", q, k) * m["scale"] * p("temp")[:, None, None]
    mask = m.get("mask") or {}
    w = sink_softmax(scores, seen_keys(T, mask.get("size"), mask.get("keep_first")), p("sink"))
    o = turn_pairs(torch.einsum("hij,jhd->ihd", w, v), pos, vfreq, sign=-1.0)
    return (o.reshape(T, H * dv) * torch.sigmoid(h @ p("g").T)) @ p("o").T


def latent_attention(h, p, m, eps):
    """Queries through a small normed vector, keys and values of every head from another one; nothing is turned; a window
    and a sink."""
    T = h.shape[0]
    H, dk, dv = m["heads"], m["dim"], m["vdim"]
    q = (rms_norm(h @ p("dq").T, p("dq.norm"), eps) @ p("uq").T).view(T, H, dk)
    c = rms_norm(h @ p("dkv").T, p("dkv.norm"), eps)
    k = (c @ p("uk").T).view(T, H, dk)
    v = (c @ p("uv").T).view(T, H, dv)
    mask = m.get("mask") or {}
    scores = torch.einsum("ihd,jhd->hij", q, k) * m["scale"]
    w = sink_softmax(scores, seen_keys(T, mask.get("size"), mask.get("keep_first")), p("sink"))
    return torch.einsum("hij,jhd->ihd", w, v).reshape(T, H * dv) @ p("o").T


# ----------------------------------------------------------------------------
# feed-forwards
# ----------------------------------------------------------------------------

def poly_norm(z, numbers, eps):
    """The first three numbers weigh z and its (entrywise) square and cube, each divided by its own root mean square over the
    last dimension; the fourth is added to every entry."""
    return sum(numbers[k - 1] * rms_norm(z ** k, None, eps) for k in (1, 2, 3)) + numbers[3]


def dense_ff(h, p, eps):
    return poly_norm(h @ p("up").T, p("act"), eps) @ p("down").T


def expert(h, gate, up, down):
    return (silu(h @ gate.T) * (h @ up.T)) @ down.T


def moe_ff(h, p, mlp):
    """The `top` largest of W_r h + b; their weights are the softmax over these alone."""
    ro = mlp["router"]
    z = h @ p("router").T + p("router.b")
    best = z.topk(ro["top"], dim=-1)
    weights = torch.softmax(best.values, dim=-1)
    y = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, we in zip(best.indices[t].tolist(), weights[t]):
            y[t] += we * expert(h[t], p(f"e{e}.gate"), p(f"e{e}.up"), p(f"e{e}.down"))
    return y


# ----------------------------------------------------------------------------
# a stream in several copies, and the model
# ----------------------------------------------------------------------------

def sublayer(xs, p, f):
    """xs [n, T, W]: f reads sum_s in[s] x_s; with its result y, x_t becomes sum_s mix[s, t] x_s + out[t] y."""
    y = f(torch.einsum("s,stw->tw", p("in"), xs))
    return torch.einsum("sd,stw->dtw", p("mix"), xs) + p("out")[:, None, None] * y


def layer_forward(xs, i, layer, cfg, w):
    """xs [n, T, W]; without copies (`streams` absent) n is 1 and a sublayer's result is simply added."""
    eps, m, mlp = cfg["norm"]["eps"], layer["mixer"], layer.get("mlp")
    at = lambda prefix: (lambda name: w[f"l{i}.{prefix}{name}"])      # noqa: E731
    mix = {"attention": attention, "latent_attention": latent_attention}[layer["type"]]
    subs = [lambda u: mix(rms_norm(u, at("")("norm1"), eps), at("mix."), m, eps)]
    if mlp is not None:
        ff = ((lambda h: dense_ff(h, at("mlp."), eps)) if mlp["kind"] == "dense" else (lambda h: moe_ff(h, at("mlp."), mlp)))
        subs.append(lambda u: ff(rms_norm(u, at("")("norm2"), eps)))
    for q, f in enumerate(subs):
        xs = sublayer(xs, at(f"hc{q + 1}."), f) if cfg.get("streams") else xs + f(xs[0])
    return xs


def forward(tokens, cfg, w, return_layers=False):
    """tokens: list of ints -> logits [T, vocab] (and the sum of the copies behind every layer)."""
    x = w["embed"][torch.as_tensor(tokens, dtype=torch.long)]
    xs = x[None].repeat(cfg.get("streams") or 1, 1, 1)
    layers = []
    for i, layer in enumerate(cfg["layers"]):
        xs = layer_forward(xs, i, layer, cfg, w)
        layers.append(xs.sum(dim=0))
    logits = rms_norm(xs.sum(dim=0), w["final.norm"], cfg["norm"]["eps"]) @ w["embed"].T
    return (logits, layers) if return_layers else logits
