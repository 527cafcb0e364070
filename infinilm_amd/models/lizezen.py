"""Lizezen: a decoder-only model whose layers run one mixer (the matrix memory of an mLSTM; a rotary softmax attention; an attention
whose values are its projected keys, with normed queries and keys, capped scores and one gate a head) beside a feed-forward (dense, or
routed experts some of which are the identity) on the same input, which a dynamic tanh makes of the residual stream, and in which a
stretch of layers may run several times in a row with the same weights, each pass beginning with a product over the stream and the
embedding's output side by side.  This file holds everything that is specific to the design: config.json's keys, their
validation, the tensor names and the description of the model as parts.  No part and no kernel knows of it.

config.json:  architecture "Lizezen"; vocab, width; norm {eps}; layers: a list of {type, mixer: {...}, mlp: {...} | null}
    type "mlstm":        mixer {heads, dim, vdim, gate_cap}
    type "attention":    mixer {heads, kv_heads, dim, vdim, scale, rot, softcap | absent}
    type "attention_2":  mixer {heads, kv_heads, dim, vdim (= dim), scale, rot, softcap | absent}
         rot {base, dims, scaling {factor, original, fast, slow} | absent}
    mlp: {kind: "dense", ff}
       | {kind: "moe", router {experts, identity | absent, groups {count, keep} | absent, top, scale}, expert {ff}, shared {ff} | absent}
  loop: {start, stop, times} or absent: layers start .. stop-1 run `times` times in a row, each pass with caches and states of its own.
Tensors (matrices stored [out, in], biases end in ".b"): embed, head, loop.in; final.norm and l<i>.norm1, each with .b and .alpha;
  mlstm:        l<i>.mix.{q, k, v, g, o, norm}, l<i>.mix.{i, f} with .b
  attention:    l<i>.mix.{q, k, v, o}
  attention_2:  l<i>.mix.{q, k, g, o, q.norm, k.norm}
  dense:        l<i>.mlp.{up, down} with .b
  moe:          l<i>.mlp.{router, correction}, l<i>.mlp.e<j>.{gate, up, down}, l<i>.mlp.shared.{gate, up, down, sg}
"""
from __future__ import annotations

import math
from dataclasses import dataclass, field
from typing import Any, Dict, List, Optional

from ..config.errors import ConfigError
from ..config.registry import register_architecture
from ..config.spec import HeadSpec, LayerRun, LayerSpec, ModelSpec, PartSpec, RunStart
from ..parts.rotary import stretched_frequencies
from .kekevik import _need

MAX_POSITIONS = 1 << 30    # the design sets no limit: angles are formed from the position in the kernels, no table


@dataclass
class LizezenLayer:
    kind: str                           # mlstm | attention | attention_2
    mixer: Dict[str, Any]               # the checked sizes and constants of its mixer
    mlp: Optional[Dict[str, Any]]       # the same of its feed-forward, None: the layer has none


@dataclass
class LizezenConfig:
    vocab: int
    width: int
    eps: float
    layers: List[LizezenLayer]
    loop: Optional[Dict[str, int]] = None      # {start, stop, times}
    dtype: Optional[str] = "bfloat16"
    eos_token_ids: List[int] = field(default_factory=list)
    raw: Dict[str, Any] = field(default_factory=dict, repr=False)

    @classmethod
    def from_dict(cls, raw: Dict[str, Any]) -> "LizezenConfig":
        vocab, width = _need(raw, "vocab", "config", int), _need(raw, "width", "config", int)
        eps = _need(raw.get("norm"), "eps", "config 'norm'")
        if eps < 0:
            raise ConfigError(f"norm.eps must not be negative, got {eps}")
        entries = _need(raw, "layers", "config", list)
        if not entries:
            raise ConfigError("config 'layers' is empty")
        layers = []
        for i, e in enumerate(entries):
            where = f"layers[{i}]"
            kind = _need(e, "type", where, str)
            m = _need(e, "mixer", where, dict)
            mw = where + ".mixer"
            if kind == "mlstm":
                mixer = {k: _need(m, k, mw, int) for k in ("heads", "dim", "vdim")}
                mixer["gate_cap"] = _positive(m, "gate_cap", mw)
            elif kind in ("attention", "attention_2"):
                mixer = {k: _need(m, k, mw, int) for k in ("heads", "kv_heads", "dim", "vdim")}
                if mixer["heads"] % mixer["kv_heads"]:
                    raise ConfigError(f"{mw}: {mixer['heads']} heads are no multiple of {mixer['kv_heads']} kv_heads")
                if kind == "attention_2" and mixer["vdim"] != mixer["dim"]:
                    raise ConfigError(f"{mw}: values that are the keys have their size {mixer['dim']}, not {mixer['vdim']}")
                mixer["scale"] = _need(m, "scale", mw)
                mixer["softcap"] = _positive(m, "softcap", mw) if m.get("softcap") is not None else 0.0
                mixer["rot"] = _rotation(m.get("rot"), mixer["dim"], mw + ".rot")
            else:
                raise ConfigError(f"{where}: unknown layer type {kind!r} (mlstm, attention, attention_2)")
            layers.append(LizezenLayer(kind, mixer, _feed_forward(e.get("mlp"), where + ".mlp")))
        loop = raw.get("loop")
        if loop is not None:
            lw = "config 'loop'"
            times = _need(loop, "times", lw, int)
            start, stop = _whole(loop, "start", lw), _whole(loop, "stop", lw)
            if not 0 <= start < stop <= len(layers):
                raise ConfigError(f"{lw}: layers {start} .. {stop - 1} are not a stretch of the {len(layers)} layers")
            loop = {"start": start, "stop": stop, "times": times}
        return cls(vocab=vocab, width=width, eps=eps, layers=layers, loop=loop, raw=dict(raw))


def _positive(d: Dict[str, Any], key: str, where: str) -> float:
    v = _need(d, key, where)
    if v <= 0:
        raise ConfigError(f"Key '{key}' in {where} must be positive, got {v}")
    return v


def _whole(d: Dict[str, Any], key: str, where: str, default: Optional[int] = None) -> int:
    """A whole number from 0 on."""
    v = d.get(key) if isinstance(d, dict) else None
    if v is None and default is not None:
        return default
    if isinstance(v, bool) or not isinstance(v, int) or v < 0:
        raise ConfigError(f"Key '{key}' in {where} must be a whole number, got {v!r}")
    return v


def _rotation(rot: Optional[dict], dim: int, where: str) -> Dict[str, Any]:
    """{dims, base, frequencies (None: base^(-2i/dims)), magnitude}."""
    dims = _whole(rot, "dims", where, 0) if rot is not None else 0
    if dims % 2 or dims > dim:
        raise ConfigError(f"{where}: dims must be even and at most dim, got {dims}")
    out = {"dims": dims, "base": 1.0, "frequencies": None, "magnitude": 1.0}
    if not dims:
        return out
    out["base"] = _positive(rot, "base", where)
    s = rot.get("scaling")
    if s is not None:
        sw = where + ".scaling"
        factor, original, fast, slow = (_positive(s, k, sw) for k in ("factor", "original", "fast", "slow"))
        if out["base"] == 1.0:
            raise ConfigError(f"{where}: a base of 1 turns every pair alike and cannot be scaled")
        out["frequencies"] = stretched_frequencies(dims, out["base"], factor, original, fast, slow, last=dims - 1)
        out["magnitude"] = 0.1 * math.log(factor) + 1.0
    return out


def _feed_forward(mlp: Optional[dict], where: str) -> Optional[Dict[str, Any]]:
    if mlp is None:
        return None
    kind = _need(mlp, "kind", where, str)
    if kind == "dense":
        return {"kind": kind, "ff": _need(mlp, "ff", where, int)}
    if kind != "moe":
        raise ConfigError(f"{where}: unknown kind {kind!r} (dense, moe)")
    r, rw = _need(mlp, "router", where, dict), where + ".router"
    out = {"kind": kind, "experts": _need(r, "experts", rw, int), "top": _need(r, "top", rw, int), "scale": _need(r, "scale", rw),
           "identity": _whole(r, "identity", rw, 0), "ff": _need(mlp.get("expert"), "ff", where + ".expert", int),
           "shared_ff": _need(mlp["shared"], "ff", where + ".shared", int) if mlp.get("shared") is not None else 0}
    g = r.get("groups")
    total = out["experts"] + out["identity"]
    out["groups"], out["keep"] = (_need(g, "count", rw + ".groups", int), _need(g, "keep", rw + ".groups", int)) if g is not None else (1, 1)
    if total % out["groups"] or out["keep"] > out["groups"]:
        raise ConfigError(f"{rw}: {total} experts in {out['groups']} groups of which {out['keep']} are kept")
    if out["top"] > out["keep"] * (total // out["groups"]):
        raise ConfigError(f"{rw}: {out['top']} experts a token from {out['keep']} groups of {total // out['groups']}")
    return out


def _mixer_spec(layer: LizezenLayer, W: int, eps: float) -> PartSpec:
    m = layer.mixer
    if layer.kind == "mlstm":
        return PartSpec("mlstm", {"hidden_size": W, "heads": m["heads"], "dim": m["dim"], "vdim": m["vdim"], "gate_cap": m["gate_cap"],
                                  "eps": eps, "bias_suffix": "b"})
    shared = layer.kind == "attention_2"
    rot = m["rot"]
    position = PartSpec("normed_pair_rotary", {"dim": m["dim"], "value_dim": m["vdim"], "rotary_dim": rot["dims"], "theta": rot["base"],
                                               "eps": eps, "qk_norm": shared, "names": ("q.norm", "k.norm"), "half_pairs": True,
                                               "frequencies": rot["frequencies"], "magnitude": rot["magnitude"], "values_are_keys": shared})
    return PartSpec("gqa_attention", {"hidden_size": W, "num_heads": m["heads"], "num_kv_heads": m["kv_heads"], "head_dim": m["dim"],
                                      "value_dim": m["vdim"], "qkv_bias": False, "out_bias": False, "scale": m["scale"], "window": 0,
                                      "softcap": m["softcap"], "position": position, "names": ("q", "k", "v", "o"), "suffix": "",
                                      "position_prefix": "", "values_are_keys": shared, "head_gate": "g" if shared else None,
                                      "float_weights": True, "head_multiple": 16})


def _ffn_spec(f: Dict[str, Any], W: int) -> PartSpec:
    if f["kind"] == "dense":
        return PartSpec("activation_mlp", {"hidden_size": W, "intermediate_size": f["ff"], "activation": "gelu_tanh", "bias": True,
                                           "names": ("up", "down"), "suffix": "", "bias_suffix": "b", "defer_bias": True})
    return PartSpec("routed_gated_experts", {"hidden_size": W, "experts": f["experts"], "top": f["top"], "expert_ff": f["ff"],
                                             "identity": f["identity"], "groups": f["groups"], "keep": f["keep"],
                                             "weight_scale": f["scale"], "shared_ff": f["shared_ff"]})


def build_spec(cfg: LizezenConfig) -> ModelSpec:
    """embed -> runs (h = tanh norm; x += mixer(h) + feed-forward(h); before a pass of the loop x = W [x; embedding]) -> tanh norm -> head."""
    W = cfg.width
    norm = PartSpec("dynamic_tanh", {"size": W, "param_name": "", "bias_name": "b", "alpha_name": "alpha"})
    layers = []
    for i, layer in enumerate(cfg.layers):
        parts = {"norm1": norm, "mixer": _mixer_spec(layer, W, cfg.eps)}
        names = {"norm1": "norm1", "mixer": "mix"}
        if layer.mlp is not None:
            parts["ffn"], names["ffn"] = _ffn_spec(layer.mlp, W), "mlp"
        layers.append(LayerSpec(prefix=f"l{i}", arrangement="parallel_residual", parts=parts, names=names))
    # the order of runs: every run of a layer has a cache entry of its own
    n = len(layers)
    a, b, times = (cfg.loop["start"], cfg.loop["stop"], cfg.loop["times"]) if cfg.loop else (0, 0, 0)
    runs = [(i, False) for i in range(a)] + [(i, i == a) for _ in range(times) for i in range(a, b)] + [(i, False) for i in range(b, n)]
    order = [LayerRun(layer=i, cache=c, writes_cache=True, start=RunStart(project_embedding=True) if begins else None)
             for c, (i, begins) in enumerate(runs)]
    spec = ModelSpec(architecture="Lizezen", vocab_size=cfg.vocab, hidden_size=W, max_positions=MAX_POSITIONS, embed_name="embed",
                     embed_scale=1.0, layers=layers, order=order, final_norm=norm, final_norm_name="final.norm",
                     head=HeadSpec(name="head", scale=1.0, tie_to_embedding_when_missing=False, params={"param_name": ""}),
                     eos_token_ids=list(cfg.eos_token_ids), embed_params={"param_name": ""},
                     run_projection="loop.in" if cfg.loop else None)
    spec.validate()
    return spec


register_architecture(["Lizezen", "lizezen"], LizezenConfig.from_dict, build_spec)
