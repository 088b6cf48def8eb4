"""Pepapel: a decoder with a norm behind every sum, whose layers are either attention over everything before (with a
temperature that grows with the position and a soft cap on its scores) or two mixers side by side: attention in chunks behind
short convolutions, beside a delta rule with one decay per head.

config.json: `vocab`, `width`, `norm.eps`, `embedding.scale`, `postln_alpha`, `layers` (each: `type`, `mixer` with the mixer's
sizes and constants, `mlp` or null).  Optional: `q_temp` and `softcap` of an attention, `mask` and `rot` (and its `scaling`) of a
pair's attention, `groups` and `identity` of a router, `max_positions` (the engine's limit on a request's length; the
architecture itself has none).

The model: x = embed[token] * embedding.scale.  A layer, with a = postln_alpha: x <- norm1(a x + mixer(x)), then, if it has a
feed-forward, x <- norm2(a x + ff(x)).  norm1, norm2 and the final norm take the mean off and have a weight and no bias.  Behind
the last layer the final norm and the head, a matrix of its own.

Mixers: "attention" (parts.mixers.CausalSelfAttention: grouped key heads, values of a width of their own, q and k normed per
head, the temperature, the soft cap, no rotation) and "parallel" (parts.mixers.ParallelMixers over parts.mixers.ConvAttention,
tensors under `left`, and parts.recurrent.GatedDelta, tensors under `right`).  Feed-forwards: "dense" (parts.feedforward.GatedMLP
with the clamped gate and biases) and "moe" (parts.feedforward.RoutedExperts: softmax scores, a correction for the choice alone,
groups judged by their best output, weights that are the scores as they are, experts of max(W_up h, 0)^2, outputs that return
their input).
"""
from __future__ import annotations

import copy
from dataclasses import dataclass

from ..config.base import ConfigError, read_float, read_int, read_str
from ..config.registry import register_architecture
from ..parts.model import DecoderSpec, LayerCall, LayerSpec

LAYER_TYPES = ("attention", "parallel")
DEFAULT_MAX_POSITIONS = 65536
GATE_ALPHA = 1.702      # of the dense feed-forward's sigmoid, fixed by the design
UNIT_EPS = 1e-6         # under the root of the delta rule's unit vectors, likewise


def _sub(d, key, where="config.json"):
    v = d.get(key)
    if not isinstance(v, dict):
        raise ConfigError(f"{where}: key '{key}' must be an object")
    return v


def _read_heads(m, where):
    heads, kv = read_int(m, "heads", minimum=1), read_int(m, "kv_heads", minimum=1)
    if heads % kv != 0:
        raise ConfigError(f"{where}: heads ({heads}) is no multiple of kv_heads ({kv})")
    read_int(m, "dim", minimum=1), read_int(m, "vdim", minimum=1)


def _check_mixer(kind, m, where):
    if kind == "attention":
        _read_heads(m, where)
        read_float(m, "scale")
        if m.get("q_temp") is not None:
            qt = _sub(m, "q_temp", where)
            read_float(qt, "coef")
            if not read_float(qt, "every") > 0:
                raise ConfigError(f"{where}.q_temp.every = {qt['every']}: a number of positions above 0")
        if m.get("softcap") is not None and not read_float(m, "softcap") > 0:
            raise ConfigError(f"{where}.softcap = {m['softcap']}: a number above 0")
        return
    left, right = _sub(m, "left", where), _sub(m, "right", where)
    _read_heads(left, where + ".left"), _read_heads(right, where + ".right")
    read_float(left, "scale")
    read_int(left, "conv", minimum=1), read_int(right, "conv", minimum=1)
    if left.get("mask") is not None:
        read_int(_sub(left, "mask", where + ".left"), "size", minimum=1)
    if left.get("rot") is not None:
        rot = _sub(left, "rot", where + ".left")
        read_float(rot, "base")
        dims = read_int(rot, "dims", minimum=0)
        if dims % 2 or dims > left["dim"]:
            raise ConfigError(f"{where}.left.rot.dims = {dims}: an even number up to dim ({left['dim']})")
        if rot.get("scaling") is not None and not read_float(_sub(rot, "scaling", where + ".left.rot"), "factor") > 0:
            raise ConfigError(f"{where}.left.rot.scaling.factor = {rot['scaling']['factor']}: a number above 0")


def _check_mlp(mlp, where):
    if not isinstance(mlp, dict):
        raise ConfigError(f"{where} must be an object or null")
    if read_str(mlp, "kind", choices=("dense", "moe")) == "dense":
        read_int(mlp, "ff", minimum=1), read_float(mlp, "limit")
        return
    read_int(_sub(mlp, "expert", where), "ff", minimum=1)
    ro = _sub(mlp, "router", where)
    n, top = read_int(ro, "experts", minimum=1), read_int(ro, "top", minimum=1)
    n += read_int(ro, "identity", default=None, minimum=0) or 0
    groups, keep = 1, 1
    if ro.get("groups") is not None:
        gr = _sub(ro, "groups", where + ".router")
        groups, keep = read_int(gr, "count", minimum=1), read_int(gr, "keep", minimum=1)
    if n % groups or keep > groups or top > keep * (n // groups):
        raise ConfigError(f"{where}.router: {n} outputs in {groups} groups of which {keep} are kept cannot give {top} choices")


@dataclass(frozen=True)
class PepapelConfig:
    raw: dict

    architecture = "Pepapel"

    @property
    def vocab(self):
        return self.raw["vocab"]

    @property
    def width(self):
        return self.raw["width"]

    @property
    def eps(self):
        return float(self.raw["norm"]["eps"])

    @property
    def layers(self):
        return self.raw["layers"]

    @property
    def max_positions(self):
        return self.raw.get("max_positions") or DEFAULT_MAX_POSITIONS

    @classmethod
    def from_dict(cls, d: dict) -> "PepapelConfig":
        raw = copy.deepcopy({k: v for k, v in d.items() if k not in ("architectures", "torch_dtype")})
        read_int(raw, "vocab", minimum=1), read_int(raw, "width", minimum=1)
        read_float(_sub(raw, "norm"), "eps")
        read_float(_sub(raw, "embedding"), "scale")
        read_float(raw, "postln_alpha")
        read_int(raw, "max_positions", default=None, minimum=1)
        layers = raw.get("layers")
        if not isinstance(layers, list) or not layers:
            raise ConfigError("config.json: key 'layers' must be a list of layers")
        for i, layer in enumerate(layers):
            where = f"config.json: layers[{i}]"
            if not isinstance(layer, dict):
                raise ConfigError(f"{where} must be an object")
            kind = read_str(layer, "type", choices=LAYER_TYPES)
            _check_mixer(kind, _sub(layer, "mixer", where), where + ".mixer")
            if layer.get("mlp") is not None:
                _check_mlp(layer["mlp"], where + ".mlp")
        return cls(raw)

    def to_dict(self) -> dict:
        d = copy.deepcopy(self.raw)
        d["architecture"] = self.architecture
        return d


def _attention(cfg, m, p):
    H, G, dk, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    qt = m.get("q_temp")
    return ("causal_attention", dict(
        width=cfg.width, n_heads=H, n_kv_heads=G, head_dim=dk, value_dim=dv, scale=m["scale"], softcap=m.get("softcap") or 0.0,
        position_temp=(qt["coef"], qt["every"]) if qt else None, qk_norm=dict(q=p + "q.norm", k=p + "k.norm", eps=cfg.eps),
        qkv_weight=p + "q+k+v", qkv_bias=None, out_weight=p + "o", out_bias=None,
        qkv_weight_sources=((p + "q", H * dk), (p + "k", G * dk), (p + "v", G * dv))))


def _parallel(cfg, m, p):
    left, right = m["left"], m["right"]
    convs = lambda at: {s + "_conv": at + s + ".conv" for s in "qkv"}      # noqa: E731
    lp, rp = p + "left.", p + "right."
    rot = left.get("rot")
    position = dict(dims=rot["dims"], base=rot["base"], factor=float((rot.get("scaling") or {}).get("factor", 1.0))) if rot else None
    attention = ("conv_attention", dict(
        width=cfg.width, n_heads=left["heads"], n_kv_heads=left["kv_heads"], head_dim=left["dim"], value_dim=left["vdim"], taps=left["conv"],
        scale=left["scale"], eps=cfg.eps, chunk=(left.get("mask") or {}).get("size", 0), position=position,
        names=dict({s: lp + s for s in ("q", "k", "v", "g", "o")}, q_norm=lp + "q.norm", k_norm=lp + "k.norm", **convs(lp))))
    delta = ("gated_delta", dict(
        width=cfg.width, n_heads=right["heads"], n_qk_heads=right["kv_heads"], head_dim=right["dim"], value_dim=right["vdim"],
        taps=right["conv"], eps=cfg.eps, unit_eps=UNIT_EPS,
        names=dict({s: rp + s for s in ("q", "k", "v", "g", "b", "a", "o", "A_log", "dt_bias", "norm")}, **convs(rp))))
    return ("parallel_mixers", dict(width=cfg.width, eps=cfg.eps, branches=[attention, delta], norm_names=[lp + "out", rp + "out"]))


def _feed_forward(cfg, mlp, p):
    W = cfg.width
    if mlp is None:
        return ("none", {})
    if mlp["kind"] == "dense":
        return ("gated_mlp", dict(width=W, inner=mlp["ff"], activation="clamped", limit=mlp["limit"], alpha=GATE_ALPHA,
                                  gate_weight=p + "gate", up_weight=p + "up", down_weight=p + "down", gate_bias=p + "gate.b",
                                  up_bias=p + "up.b", down_bias=p + "down.b"))
    ro = mlp["router"]
    groups = ro.get("groups") or {"count": 1, "keep": 1}
    return ("routed_experts", dict(
        width=W, inner=mlp["expert"]["ff"], n_experts=ro["experts"], top=ro["top"], router=p + "router", correction=p + "correction",
        gate=None, up=p + "e{e}.up", down=p + "e{e}.down", score="softmax", renorm=False, act="relu2", groups=groups["count"],
        keep=groups["keep"], group_by="best", identity=ro.get("identity") or 0))


def build_pepapel(cfg: PepapelConfig) -> DecoderSpec:
    W = cfg.width

    def norm(name):
        return ("layernorm_of_sum", dict(width=W, eps=cfg.eps, weight_name=name, alpha=float(cfg.raw["postln_alpha"])))
    layers, order, caches = [], [], 0
    for i, layer in enumerate(cfg.layers):
        p = f"l{i}."
        mixer = (_attention if layer["type"] == "attention" else _parallel)(cfg, layer["mixer"], p + "mix.")
        layers.append(LayerSpec(arrangement="post_norm", parts=dict(
            mixer=mixer, norm1=norm(p + "norm1"), ffn=_feed_forward(cfg, layer.get("mlp"), p + "mlp."), norm2=norm(p + "norm2"))))
        # (a pair: pages, the convolution's last rows if it has more than one tap, the delta rule's state)
        k = 1 if layer["type"] == "attention" else 3 if layer["mixer"]["left"]["conv"] > 1 else 2
        order.append(LayerCall(layer=i, cache=tuple(range(caches, caches + k)) if k > 1 else caches))
        caches += k
    return DecoderSpec(
        vocab=cfg.vocab, width=W, max_positions=cfg.max_positions, token_table="embed", position=("none", {}),
        layers=layers, run_order=order, final_norm=("layernorm", dict(width=W, eps=cfg.eps, weight_name="final.norm", bias_name=None)),
        head_weight="head", embedding_scale=float(cfg.raw["embedding"]["scale"]),
        # (a layer without a feed-forward has no use for its second norm, whether or not a file holds it)
        ignore_tensors=tuple(rf"^l{i}\.norm2$" for i, layer in enumerate(cfg.layers) if layer.get("mlp") is None))


register_architecture(["Pepapel"], PepapelConfig, build_pepapel)
