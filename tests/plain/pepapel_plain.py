"""A plain, slow Pepapel: whole sequences, no cache, one function per mechanism.

It shares no code with the engine.  Every function works on one sequence, [tokens, ...] torch tensors on
the CPU, in the precision of the tensors it is given (float32, or float64 to see how much of a
difference is rounding).  Weights come as a dict from tensor name to tensor; `cfg` is config.json as a
dict.

Notation: T tokens, W the model's width, H heads, G heads of keys (and, in the delta rule, of queries) where they are
fewer, dk and dv a head's key and value sizes; `p(name)` is a layer's tensor.
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


def layer_norm(x, weight, eps):
    """The mean taken off, divided by the root of the mean squared deviation (plus eps), weighed."""
    d = x - x.mean(dim=-1, keepdim=True)
    return d / torch.sqrt((d * d).mean(dim=-1, keepdim=True) + eps) * weight


def silu(z):
    return z * torch.sigmoid(z)


def softplus(z):
    return torch.log1p(torch.exp(-z.abs())) + torch.clamp(z, min=0)


def causal_taps(x, w):
    """x [T, C], w [C, taps]: y_t = sum_j w[:, j] x_(t - taps + 1 + j), the last column weighs the token itself;
    nothing before the first token."""
    T, taps = x.shape[0], w.shape[1]
    y = torch.zeros_like(x)
    for j in range(taps):
        back = taps - 1 - j
        if back < T:
            y[back:] += w[:, j] * x[:T - back]
    return y


def turn_halves(x, positions, rot):
    """x [T, n, d]: of each vector's first `dims` entries, entry i and entry i + dims / 2 are turned by the angle
    position * base^(-2i/dims) / factor; the rest stay."""
    out = x.clone()
    if not rot or not rot["dims"]:
        return out
    half = rot["dims"] // 2
    factor = float((rot.get("scaling") or {}).get("factor", 1.0))
    f = torch.tensor([float(rot["base"]) ** (-2.0 * i / rot["dims"]) / factor for i in range(half)], dtype=torch.float64)
    ang = positions.to(torch.float64)[:, None] * f[None, :]
    cos, sin = torch.cos(ang).to(x.dtype)[:, None, :], torch.sin(ang).to(x.dtype)[:, None, :]
    u, v = x[..., :half], x[..., half:2 * half]
    out[..., :half] = u * cos - v * sin
    out[..., half:2 * half] = v * cos + u * sin
    return out


def softmax_read(scores, seen, v):
    """scores [H, T, T] (query, key), v [T, H, dv] -> [T, H, dv]"""
    w = torch.softmax(scores.masked_fill(~seen, float("-inf")), dim=-1)
    return torch.einsum("hij,jhd->ihd", w, v)


def causal_mask(T, chunk=None):
    """[T, T] (query i, key j): j <= i, and, with chunks, in the same run of `chunk` positions."""
    i, j = torch.arange(T)[:, None], torch.arange(T)[None, :]
    seen = j <= i
    return seen & (i // chunk == j // chunk) if chunk else seen


# ----------------------------------------------------------------------------
# mixers
# ----------------------------------------------------------------------------

def query_temperature(positions, q_temp):
    """1 + coef ln(floor((position + 1) / every) + 1), a number per position."""
    if not q_temp:
        return torch.ones(len(positions), dtype=torch.float64)
    return torch.tensor([1.0 + q_temp["coef"] * math.log(math.floor((int(p) + 1) / q_temp["every"]) + 1.0) for p in positions],
                        dtype=torch.float64)


def capped_attention(h, p, m, eps):
    """Queries and keys normed per head, queries times a temperature of their position, scores through a soft cap."""
    T = h.shape[0]
    H, G, dk, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = rms_norm((h @ p("q").T).view(T, H, dk), p("q.norm"), eps)
    k = rms_norm((h @ p("k").T).view(T, G, dk), p("k.norm"), eps).repeat_interleave(H // G, dim=1)
    v = (h @ p("v").T).view(T, G, dv).repeat_interleave(H // G, dim=1)
    q = q * query_temperature(range(T), m.get("q_temp")).to(h.dtype)[:, None, None]
    s = torch.einsum("ihd,jhd->hij", q, k) * m["scale"]
    if m.get("softcap"):
        s = m["softcap"] * torch.tanh(s / m["softcap"])
    return softmax_read(s, causal_mask(T), v).reshape(T, H * dv) @ p("o").T


def conv_attention(h, p, m, eps):
    """Queries, keys and values through a short convolution; queries and keys normed over all heads at once and turned by
    the position; chunks; a gate per head."""
    T = h.shape[0]
    H, G, dk, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k, v = (causal_taps(h @ p(s).T, p(s + ".conv")) for s in "qkv")
    q, k = rms_norm(q, p("q.norm"), eps), rms_norm(k, p("k.norm"), eps)
    pos = torch.arange(T)
    q = turn_halves(q.view(T, H, dk), pos, m.get("rot"))
    k = turn_halves(k.view(T, G, dk), pos, m.get("rot")).repeat_interleave(H // G, dim=1)
    v = v.view(T, G, dv).repeat_interleave(H // G, dim=1)
    s = torch.einsum("ihd,jhd->hij", q, k) * m["scale"]
    o = softmax_read(s, causal_mask(T, (m.get("mask") or {}).get("size")), v)
    return (o * torch.sigmoid(h @ p("g").T)[:, :, None]).reshape(T, H * dv) @ p("o").T


def gated_delta(h, p, m, eps):
    """The delta rule with one decay per head and token.  q and k (G heads) and v (H heads) pass a short convolution and
    silu; q and k become unit vectors, q times dim^(-1/2).  Per head: S <- g S; u = beta (v - S^T k); S <- S + k u^T;
    o = S^T q.  Each head's o over its root mean square, weighed, times silu of a gate."""
    T = h.shape[0]
    H, G, dk, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k, v = (silu(causal_taps(h @ p(s).T, p(s + ".conv"))) for s in "qkv")
    q, k, v = q.view(T, G, dk), k.view(T, G, dk), v.view(T, H, dv)
    q = q / torch.sqrt((q * q).sum(-1, keepdim=True) + 1e-6) * dk ** -0.5
    k = k / torch.sqrt((k * k).sum(-1, keepdim=True) + 1e-6)
    q, k = q.repeat_interleave(H // G, dim=1), k.repeat_interleave(H // G, dim=1)
    beta = torch.sigmoid(h @ p("b").T)                                                   # [T, H]
    g = torch.exp(-torch.exp(p("A_log")) * softplus(h @ p("a").T + p("dt_bias")))        # [T, H]
    S = torch.zeros(H, dk, dv, dtype=h.dtype)
    o = torch.zeros(T, H, dv, dtype=h.dtype)
    for t in range(T):
        S = g[t][:, None, None] * S
        u = beta[t][:, None] * (v[t] - torch.einsum("hkv,hk->hv", S, k[t]))
        S = S + k[t][:, :, None] * u[:, None, :]
        o[t] = torch.einsum("hkv,hk->hv", S, q[t])
    y = rms_norm(o, p("norm"), eps) * silu(h @ p("g").T).view(T, H, dv)
    return y.reshape(T, H * dv) @ p("o").T


def parallel(h, p, m, eps):
    left = conv_attention(h, lambda s: p("left." + s), m["left"], eps)
    right = gated_delta(h, lambda s: p("right." + s), m["right"], eps)
    return 0.5 * (rms_norm(left, p("left.out"), eps) + rms_norm(right, p("right.out"), eps))


# ----------------------------------------------------------------------------
# feed-forwards
# ----------------------------------------------------------------------------

def dense_ff(h, p, mlp):
    g = torch.clamp(h @ p("gate").T + p("gate.b"), max=mlp["limit"])
    u = torch.clamp(h @ p("up").T + p("up.b"), min=-mlp["limit"], max=mlp["limit"])
    return (g * torch.sigmoid(1.702 * g) * (u + 1)) @ p("down").T + p("down.b")


def choose(s, correction, router):
    """s [n] -> the chosen outputs' numbers.  Runs of neighbours compete first, each with its best s + correction."""
    c = s if correction is None else s + correction
    groups = router.get("groups") or {"count": 1, "keep": 1}
    runs = c.view(groups["count"], -1)
    kept = torch.topk(runs.max(dim=1).values, groups["keep"]).indices
    open_ = torch.full_like(runs, float("-inf"))
    open_[kept] = runs[kept]
    return torch.topk(open_.reshape(-1), router["top"]).indices


def moe_ff(h, p, mlp, correction):
    """The router has `experts` + `identity` outputs; a chosen output beyond the experts gives the token's row back."""
    ro = mlp["router"]
    s = torch.softmax(h @ p("router").T, dim=-1)
    y = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e in choose(s[t], correction, ro).tolist():
            out = h[t]
            if e < ro["experts"]:
                out = torch.clamp(h[t] @ p(f"e{e}.up").T, min=0) ** 2 @ p(f"e{e}.down").T
            y[t] += s[t, e] * out
    return y


# ----------------------------------------------------------------------------
# the model
# ----------------------------------------------------------------------------

def layer_forward(x, i, layer, cfg, w):
    eps, alpha, m, mlp = cfg["norm"]["eps"], cfg["postln_alpha"], layer["mixer"], layer.get("mlp")
    at = lambda prefix: (lambda name: w[f"l{i}.{prefix}{name}"])      # noqa: E731
    mix = {"attention": capped_attention, "parallel": parallel}[layer["type"]]
    x = layer_norm(alpha * x + mix(x, at("mix."), m, eps), w[f"l{i}.norm1"], eps)
    if mlp is not None:
        y = dense_ff(x, at("mlp."), mlp) if mlp["kind"] == "dense" else moe_ff(x, at("mlp."), mlp, w.get(f"l{i}.mlp.correction"))
        x = layer_norm(alpha * x + y, w[f"l{i}.norm2"], eps)
    return x


def forward(tokens, cfg, w, return_layers=False):
    """tokens: list of ints -> logits [T, vocab] (and the stream behind every layer)."""
    x = w["embed"][torch.as_tensor(tokens, dtype=torch.long)] * cfg["embedding"]["scale"]
    layers = []
    for i, layer in enumerate(cfg["layers"]):
        x = layer_forward(x, i, layer, cfg, w)
        layers.append(x)
    logits = layer_norm(x, w["final.norm"], cfg["norm"]["eps"]) @ w["head"].T
    return (logits, layers) if return_layers else logits
