"""Fikupel: a decoder whose layers are attention in a sliding window that keeps the first tokens, or latent attention in a
sliding window, on a stream that is kept as several copies.

config.json: `vocab`, `width`, `norm.eps`, `layers` (each: `type`, `mixer` with the mixer's sizes and constants, `mlp` or null).
Optional: `streams` (the number of copies of the stream; absent: one stream with plain residual sums), a mixer's `mask` (absent:
every key is read), an attention's `mask.keep_first`, `rot` and `rot.scaling`, and `max_positions` (the engine's limit on a
request's length; the architecture itself has none).

The model: x = embed[token], which every copy x_1 .. x_n starts as.  For sublayer q of a layer (1: the mixer, 2: the
feed-forward, if there is one), with the layer's tensors hc<q>.in / out / mix: u = sum_s in[s] x_s; y = sublayer(norm<q>(u));
x_t <- sum_s mix[s, t] x_s + out[t] y for all t at once.  Behind the last layer x is the sum of the copies; the model's norm, and
the logits are embed x.  All norms are x / sqrt(mean(x^2) + eps) * w.

Mixers: "attention" (parts.mixers.CausalSelfAttention: q and k normed per head with shared weights, part of each head turned by
the position with a stretched encoding, values turned over their whole width and the result turned back, scores times a number per
head, a window with kept first tokens, a sink per head, a gate per entry) and "latent_attention" (parts.mixers.LatentAttention
with queries through a small vector too, nothing turned, a window and a sink per head).  Feed-forwards: "dense"
(parts.feedforward.DenseMLP with the polynomial of normed powers) and "moe" (parts.feedforward.RoutedExperts: a router with a
bias, the softmax over the chosen logits, silu-gated experts).
"""
from __future__ import annotations

import copy
from dataclasses import dataclass

from ..config.base import ConfigError, read_float, read_int, read_str
from ..config.registry import register_architecture
from ..parts.model import DecoderSpec, LayerCall, LayerSpec

MIXER_TYPES = ("attention", "latent_attention")
DEFAULT_MAX_POSITIONS = 65536


def _sub(d, key, where="config.json"):
    v = d.get(key)
    if not isinstance(v, dict):
        raise ConfigError(f"{where}: key '{key}' must be an object")
    return v


def _check_mask(m, where, keeps):
    mask = m.get("mask")
    if mask is None:
        return
    mask = _sub(m, "mask", where)
    read_int(mask, "size", minimum=1)
    keep = read_int(mask, "keep_first", default=0, minimum=0)
    if keep and not keeps:
        raise ConfigError(f"{where}.mask.keep_first: this mixer's window keeps no first tokens")


def _check_rot(m, where, dim, vdim):
    rot = m.get("rot")
    if rot is None:
        return
    rot = _sub(m, "rot", where)
    dims = read_int(rot, "dims", minimum=0)
    if dims % 2 or dims > dim:
        raise ConfigError(f"{where}.rot.dims = {dims}: an even number of a head's {dim} dimensions")
    if read_float(rot, "base") <= 1:
        raise ConfigError(f"{where}.rot.base = {rot['base']}: it must be above 1")
    if vdim % 2:
        raise ConfigError(f"{where}.vdim = {vdim}: values are turned in pairs")
    if rot.get("scaling") is not None:
        sc = _sub(rot, "scaling", where + ".rot")
        for key in ("factor", "low", "high", "original"):
            if read_float(sc, key) <= 0:
                raise ConfigError(f"{where}.rot.scaling.{key} = {sc[key]}: it must be above 0")
        if sc["high"] < sc["low"]:
            raise ConfigError(f"{where}.rot.scaling: high ({sc['high']}) is below low ({sc['low']})")


def _check_layer(i, layer):
    where = f"config.json: layers[{i}]"
    if not isinstance(layer, dict):
        raise ConfigError(f"{where} must be an object")
    kind = read_str(layer, "type", choices=MIXER_TYPES)
    m, wm = _sub(layer, "mixer", where), where + ".mixer"
    heads, dim, vdim = (read_int(m, key, minimum=1) for key in ("heads", "dim", "vdim"))
    read_float(m, "scale")
    _check_mask(m, wm, kind == "attention")
    if kind == "attention":
        kv = read_int(m, "kv_heads", minimum=1)
        if heads % kv != 0:
            raise ConfigError(f"{wm}: heads ({heads}) is no multiple of kv_heads ({kv})")
        _check_rot(m, wm, dim, vdim)
    else:
        read_int(m, "kv_rank", minimum=1), read_int(m, "q_rank", minimum=1)
    mlp = layer.get("mlp")
    if mlp is None:
        return
    if not isinstance(mlp, dict):
        raise ConfigError(f"{where}.mlp must be an object or null")
    if read_str(mlp, "kind", choices=("dense", "moe")) == "dense":
        read_int(mlp, "ff", minimum=1)
    else:
        read_int(_sub(mlp, "expert", where + ".mlp"), "ff", minimum=1)
        ro = _sub(mlp, "router", where + ".mlp")
        n, top = read_int(ro, "experts", minimum=1), read_int(ro, "top", minimum=1)
        if top > n:
            raise ConfigError(f"{where}.mlp.router: {top} of {n} experts")


@dataclass(frozen=True)
class FikupelConfig:
    raw: dict

    architecture = "Fikupel"

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
    def streams(self):
        return self.raw.get("streams") or 0

    @property
    def max_positions(self):
        return self.raw.get("max_positions") or DEFAULT_MAX_POSITIONS

    @classmethod
    def from_dict(cls, d: dict) -> "FikupelConfig":
        raw = copy.deepcopy({k: v for k, v in d.items() if k not in ("architectures", "torch_dtype")})
        read_int(raw, "vocab", minimum=1), read_int(raw, "width", minimum=1)
        read_float(_sub(raw, "norm"), "eps")
        read_int(raw, "streams", default=None, minimum=1)
        read_int(raw, "max_positions", default=None, minimum=1)
        layers = raw.get("layers")
        if not isinstance(layers, list) or not layers:
            raise ConfigError("config.json: key 'layers' must be a list of layers")
        for i, layer in enumerate(layers):
            _check_layer(i, layer)
        return cls(raw)

    def to_dict(self) -> dict:
        d = copy.deepcopy(self.raw)
        d["architecture"] = self.architecture
        return d


def _mixer(cfg: FikupelConfig, i: int, layer: dict):
    m, p, W = layer["mixer"], f"l{i}.mix.", cfg.width
    mask = m.get("mask") or {}
    window = mask.get("size", 0)
    if layer["type"] == "latent_attention":
        names = {s: p + s for s in ("dq", "uq", "dkv", "uk", "uv", "sink", "o")}
        names.update(dq_norm=p + "dq.norm", dkv_norm=p + "dkv.norm")
        return ("latent_attention", dict(
            width=W, n_heads=m["heads"], head_dim=m["dim"], rot_dim=0, value_dim=m["vdim"], kv_rank=m["kv_rank"], q_rank=m["q_rank"],
            scale=m["scale"], eps=cfg.eps, window=window, position=None, names=names))
    H, G, dk, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    rot = m.get("rot")
    return ("causal_attention", dict(
        width=W, n_heads=H, n_kv_heads=G, head_dim=dk, value_dim=dv, scale=m["scale"], window=window, keep_first=mask.get("keep_first", 0),
        qkv_weight=p + "q+k+v+g", qkv_bias=None, out_weight=p + "o", out_bias=None,
        qkv_weight_sources=((p + "q", H * dk), (p + "k", G * dk), (p + "v", G * dv)), entry_gate=p + "g", sink=p + "sink", temp=p + "temp",
        qk_norm=dict(q=p + "q.norm", k=p + "k.norm", eps=cfg.eps), turn_values=rot is not None,
        position=("rotary_pairs", dict(dims=rot["dims"], base=rot["base"], head_dim=dk, scaling=rot.get("scaling"))) if rot else None))


def _feed_forward(cfg: FikupelConfig, i: int, mlp):
    p, W = f"l{i}.mlp.", cfg.width
    if mlp is None:
        return ("none", {})
    if mlp["kind"] == "dense":
        return ("dense_mlp", dict(width=W, inner=mlp["ff"], activation="poly_norm", activation_params=p + "act", eps=cfg.eps,
                                  up_weight=p + "up", up_bias=None, down_weight=p + "down", down_bias=None))
    ro = mlp["router"]
    return ("routed_experts", dict(
        width=W, inner=mlp["expert"]["ff"], n_experts=ro["experts"], top=ro["top"], router=p + "router", router_bias=p + "router.b",
        correction=None, gate=p + "e{e}.gate", up=p + "e{e}.up", down=p + "e{e}.down", score="softmax", renorm=True, weigh="output",
        act="silu"))


def build_fikupel(cfg: FikupelConfig) -> DecoderSpec:
    W, n = cfg.width, cfg.streams

    def norm(name):
        return ("rmsnorm", dict(width=W, eps=cfg.eps, weight_name=name))

    layers, ignore = [], []
    for i, layer in enumerate(cfg.layers):
        p = f"l{i}."
        parts = dict(norm1=norm(p + "norm1"), mixer=_mixer(cfg, i, layer), norm2=norm(p + "norm2"), ffn=_feed_forward(cfg, i, layer.get("mlp")))
        if n:
            for q in ("hc1", "hc2"):
                parts[q] = ("stream_mixer", dict(n_streams=n, in_name=f"{p}{q}.in", out_name=f"{p}{q}.out", mix_name=f"{p}{q}.mix"))
        if layer.get("mlp") is None:      # (no use for the second sublayer's tensors, whether or not a file holds them)
            ignore.append(rf"^l{i}\.(norm2|hc2\.(in|out|mix))$")
        layers.append(LayerSpec(arrangement="multi_stream" if n else "pre_norm_plain", parts=parts))
    return DecoderSpec(
        vocab=cfg.vocab, width=W, max_positions=cfg.max_positions, token_table="embed", position=("none", {}), layers=layers,
        run_order=[LayerCall(layer=i, cache=i) for i in range(len(layers))], final_norm=norm("final.norm"), streams=n,
        ignore_tensors=tuple(ignore))


register_architecture(["Fikupel"], FikupelConfig, build_fikupel)
