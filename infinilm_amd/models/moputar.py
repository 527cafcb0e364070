"""Moputar: a decoder-only model whose residual stream runs in several copies that every sublayer reads and writes through
small weights of its own, with two mixers a layer may pick (a gated delta rule with short convolutions; an attention inside
chunks of positions with short convolutions, norms over whole query and key rows and rotated pairs, which may read another
layer's keys and values) and a gelu-gated feed-forward a layer may lack.  This file holds everything that is specific to the
design: config.json's keys, their validation, the tensor names and the description of the model as parts.  No part and no
kernel knows of it.

config.json:  architecture "Moputar"; vocab, width; streams; embedding {scale}; norm {eps}; layers: a list of {type, mixer, mlp}
    type "delta":      mixer {heads, kv_heads, dim, vdim, conv (taps; absent: no convolution)}
    type "attention":  mixer {heads, kv_heads, dim, vdim, scale, conv (absent: none), rot {base, dims} | absent,
                              mask {size} | absent, kv_from: j | absent}
    mlp: null | {kind: "dense", ff}
Tensors (matrices stored [out, in]): embed, head, final.norm; l<i>.norm1, l<i>.norm2 (norm weights lie around zero);
  l<i>.hc1.{in, out, mix}, l<i>.hc2.{in, out, mix};
  delta:      l<i>.mix.{q, k, v} with .conv, l<i>.mix.{b, a, g, A_log, dt_bias, norm, o}
  attention:  l<i>.mix.{q, k, v} with .conv, q.norm, k.norm, o      (no k, v tensors with kv_from)
  dense:      l<i>.mlp.{gate, up, down}
"""
from __future__ import annotations

from dataclasses import dataclass, field
from typing import Any, Dict, List, Optional

from ..config.errors import ConfigError
from ..config.registry import register_architecture
from ..config.spec import HeadSpec, LayerRun, LayerSpec, ModelSpec, PartSpec
from .kekevik import _need

MAX_POSITIONS = 1 << 30      # the design sets no limit: angles are formed from the position in the kernels, no table


@dataclass
class MoputarLayer:
    kind: str                    # delta | attention
    mixer: Dict[str, Any]        # the checked sizes and constants of its mixer
    ff: Optional[int]            # the feed-forward's inner size, None: the layer has none


@dataclass
class MoputarConfig:
    vocab: int
    width: int
    streams: int
    embedding_scale: float
    eps: float
    layers: List[MoputarLayer]
    dtype: Optional[str] = "bfloat16"
    eos_token_ids: List[int] = field(default_factory=list)
    raw: Dict[str, Any] = field(default_factory=dict, repr=False)

    @classmethod
    def from_dict(cls, raw: Dict[str, Any]) -> "MoputarConfig":
        vocab, width, streams = (_need(raw, k, "config", int) for k in ("vocab", "width", "streams"))
        emb = raw.get("embedding")
        scale = _need(emb, "scale", "config 'embedding'") if emb is not None and emb.get("scale") is not None else 1.0
        eps = _need(raw.get("norm"), "eps", "config 'norm'")
        if eps < 0:
            raise ConfigError(f"norm.eps must not be negative, got {eps}")
        entries = _need(raw, "layers", "config", list)
        if not entries:
            raise ConfigError("config 'layers' is empty")
        layers: List[MoputarLayer] = []
        for i, e in enumerate(entries):
            where = f"layers[{i}]"
            kind = _need(e, "type", where, str)
            m = _need(e, "mixer", where, dict)
            mw = where + ".mixer"
            if kind not in ("delta", "attention"):
                raise ConfigError(f"{where}: unknown layer type {kind!r} (delta, attention)")
            mixer = {k: _need(m, k, mw, int) for k in ("heads", "kv_heads", "dim", "vdim")}
            if mixer["heads"] % mixer["kv_heads"]:
                raise ConfigError(f"{mw}: {mixer['heads']} heads do not divide into {mixer['kv_heads']} kv_heads")
            mixer["conv"] = _need(m, "conv", mw, int) if m.get("conv") is not None else 0
            if kind == "attention":
                mixer["scale"] = _need(m, "scale", mw)
                mixer["rot"] = _rot(m.get("rot"), mixer["dim"], mw + ".rot")
                mask = m.get("mask")
                mixer["chunk"] = _need(mask, "size", mw + ".mask", int) if mask is not None and mask.get("size") is not None else 0
                mixer["kv_from"] = _source(m.get("kv_from"), i, mixer, layers, mw)
            mlp = e.get("mlp")
            ff = None
            if mlp is not None:
                if _need(mlp, "kind", where + ".mlp", str) != "dense":
                    raise ConfigError(f"{where}.mlp: unknown kind {mlp['kind']!r} (dense)")
                ff = _need(mlp, "ff", where + ".mlp", int)
            layers.append(MoputarLayer(kind, mixer, ff))
        return cls(vocab=vocab, width=width, streams=streams, embedding_scale=scale, eps=eps, layers=layers, raw=dict(raw))


def _rot(rot, dim: int, where: str) -> Dict[str, Any]:
    if rot is None:
        return {"dims": 0, "base": 1.0}
    dims = rot.get("dims")
    if isinstance(dims, bool) or not isinstance(dims, int) or dims < 0 or dims % 2 or dims > dim:
        raise ConfigError(f"Key 'dims' in {where} must be an even number of at most the head's {dim} entries, got {dims!r}")
    return {"dims": dims, "base": _need(rot, "base", where)}


def _source(src, i: int, mixer: Dict[str, Any], layers: List[MoputarLayer], where: str) -> Optional[int]:
    """The layer whose keys and values layer i reads, or None for its own."""
    if src is None:
        return None
    if isinstance(src, bool) or not isinstance(src, int) or not 0 <= src < i:
        raise ConfigError(f"{where}: kv_from must name an earlier layer, got {src!r}")
    other = layers[src]
    if other.kind != "attention" or other.mixer["kv_from"] is not None:
        raise ConfigError(f"{where}: kv_from names layer {src}, which has no keys and values of its own")
    for k in ("heads", "kv_heads", "dim", "vdim"):
        if other.mixer[k] != mixer[k]:
            raise ConfigError(f"{where}: '{k}' is {mixer[k]}, but layer {src}, whose keys and values it reads, has {other.mixer[k]}")
    return src


def build_spec(cfg: MoputarConfig) -> ModelSpec:
    """embed[token] * scale in every stream -> layers -> the streams' sum -> final norm -> head."""
    W = cfg.width
    norm = PartSpec("rmsnorm", {"size": W, "eps": cfg.eps, "param_name": "", "weight_offset": 1.0})
    connect = PartSpec("hyper_connection", {"streams": cfg.streams})

    # the chunks by which a cache entry's readers see its keys (one that sees all keeps all)
    readers: Dict[int, List[int]] = {}
    for i, layer in enumerate(cfg.layers):
        if layer.kind == "attention":
            src = layer.mixer["kv_from"]
            readers.setdefault(i if src is None else src, []).append(layer.mixer["chunk"])
    layers, order, entry_of = [], [], {}
    n_entries = 0
    for i, layer in enumerate(cfg.layers):
        m = layer.mixer
        borrows, has_cache = None, True
        if layer.kind == "attention":
            src = m["kv_from"]
            chunks = readers[i if src is None else src]
            mixer = PartSpec("conv_attention", {
                "hidden_size": W, "heads": m["heads"], "kv_heads": m["kv_heads"], "dim": m["dim"], "vdim": m["vdim"], "scale": m["scale"],
                "eps": cfg.eps, "chunk": m["chunk"], "cache_chunks": () if 0 in chunks else tuple(sorted(set(chunks))),
                "conv_taps": m["conv"], "rotary_dim": m["rot"]["dims"], "theta": m["rot"]["base"], "own_kv": src is None})
            if src is not None:
                borrows, has_cache = entry_of[src], m["conv"] > 1
        else:
            mixer = PartSpec("gated_delta_rule", {"hidden_size": W, "heads": m["heads"], "kv_heads": m["kv_heads"], "dim": m["dim"],
                                                  "vdim": m["vdim"], "conv_taps": m["conv"], "eps": cfg.eps})
        parts = {"norm1": norm, "connect1": connect, "mixer": mixer}
        names = {"norm1": "norm1", "connect1": "hc1", "mixer": "mix"}
        if layer.ff is not None:
            parts.update(norm2=norm, connect2=connect,
                         ffn=PartSpec("gated_mlp", {"hidden_size": W, "intermediate_size": layer.ff, "activation": "gelu_tanh", "bias": False,
                                                    "names": ("gate", "up", "down"), "suffix": ""}))
            names.update(norm2="norm2", connect2="hc2", ffn="mlp")
        layers.append(LayerSpec(prefix=f"l{i}", arrangement="hyper_connected", parts=parts, names=names))
        entry = None
        if has_cache:
            entry = entry_of[i] = n_entries
            n_entries += 1
        order.append(LayerRun(layer=i, cache=entry, writes_cache=True, borrows=borrows))
    spec = ModelSpec(architecture="Moputar", vocab_size=cfg.vocab, hidden_size=W, max_positions=MAX_POSITIONS, embed_name="",
                     embed_scale=cfg.embedding_scale, layers=layers, order=order, final_norm=norm, final_norm_name="final.norm",
                     head=HeadSpec(name="head", scale=1.0, tie_to_embedding_when_missing=False, params={"param_name": ""}),
                     eos_token_ids=list(cfg.eos_token_ids), embed_params={"param_name": "embed"}, streams=cfg.streams)
    spec.validate()
    return spec


register_architecture(["Moputar", "moputar"], MoputarConfig.from_dict, build_spec)
