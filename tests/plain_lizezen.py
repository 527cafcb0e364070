"""A plain, slow implementation of the Lizezen design: whole sequences at once where a mechanism allows it, token by
token where it carries a state, one function per mechanism, in torch on the CPU (float64 unless told otherwise).  It
shares no code with the engine and is what the tests compare the engine with.

Notation: h is a sublayer's input row, p a token's position in its sequence (from 0), W x a stored [out, in] matrix
applied to a column.  `cfg` is config.json as a dict, `w` the tensors by name.
"""
from __future__ import annotations

import math
from typing import Dict, List, Optional

import torch

_ROUND = [None]     # a dtype to which every projection's operands and result are rounded (see `forward`), or None
_FORCED = [None]    # an iterator over the experts every routed feed-forward is made to choose, or None
_CHOSEN = [None]    # a list that receives the experts every routed feed-forward chose, or None


def rounded(x: torch.Tensor) -> torch.Tensor:
    return x if _ROUND[0] is None else x.to(_ROUND[0]).to(x.dtype)


def proj(h: torch.Tensor, w: torch.Tensor, b: Optional[torch.Tensor] = None) -> torch.Tensor:
    """W h (+ b) for every row of h."""
    y = rounded(h) @ w.T
    return rounded(y if b is None else y + b)


def dynamic_tanh(x: torch.Tensor, w: Dict[str, torch.Tensor], name: str) -> torch.Tensor:
    """One number scales the row before the tanh; no mean and no variance."""
    return torch.tanh(w[name + ".alpha"] * x) * w[name] + w[name + ".b"]


def rms_unit(x: torch.Tensor, eps: float) -> torch.Tensor:
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def sigmoid(x: torch.Tensor) -> torch.Tensor:
    return 1.0 / (1.0 + torch.exp(-x))


def silu(x: torch.Tensor) -> torch.Tensor:
    return x * sigmoid(x)


def log_sigmoid(x: torch.Tensor) -> torch.Tensor:
    return -(torch.log1p(torch.exp(-x.abs())) + torch.clamp(-x, min=0.0))


def gelu_tanh(z: torch.Tensor) -> torch.Tensor:
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


# ---- rotation ----------------------------------------------------------------------------------------------------------
def frequencies(rot: dict) -> List[float]:
    """The turning rates of the dims / 2 pairs, in Python floats; with 'scaling' the slow ones are stretched: pair i turns
    L f_i / (2 pi) times within the original length L, and from `fast` turns down to `slow` turns a ramp over i leads from
    f_i to f_i / factor."""
    dims, base = rot["dims"], float(rot["base"])
    f = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
    s = rot.get("scaling")
    if s is None:
        return f

    def pair_of(turns):
        return dims * math.log(s["original"] / (2.0 * math.pi * turns)) / (2.0 * math.log(base))

    lo = max(math.floor(pair_of(s["fast"])), 0)
    hi = min(math.ceil(pair_of(s["slow"])), dims - 1)
    out = []
    for i, x in enumerate(f):
        r = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(x / s["factor"] * r + x * (1.0 - r))
    return out


def magnitude(rot: dict) -> float:
    s = rot.get("scaling")
    return 1.0 if s is None else 0.1 * math.log(s["factor"]) + 1.0


def rotate_halves(x: torch.Tensor, pos: torch.Tensor, rot: Optional[dict]) -> torch.Tensor:
    """x [T, heads, dim], pos [T]: entry i turns with entry i + dims / 2 by pos * f_i; entries from `dims` on pass."""
    if not rot or not rot.get("dims"):
        return x
    n = rot["dims"] // 2
    ang = pos.to(x.dtype)[:, None] * torch.tensor(frequencies(rot), dtype=torch.float64).to(x.dtype)[None, :]
    c, s = (torch.cos(ang) * magnitude(rot))[:, None, :], (torch.sin(ang) * magnitude(rot))[:, None, :]
    out = x.clone()
    u, v = x[..., :n], x[..., n:2 * n]
    out[..., :n] = u * c - v * s
    out[..., n:2 * n] = v * c + u * s
    return out


# ---- mixers ------------------------------------------------------------------------------------------------------------
def causal_softmax(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, m: dict) -> torch.Tensor:
    """q [T, H, dim], k [T, G, dim], v [T, G, dv] -> [T, H, dv]."""
    T, H = q.shape[:2]
    per = H // k.shape[1]
    late = torch.arange(T)[None, :] > torch.arange(T)[:, None]
    out = []
    for g in range(H):
        s = (q[:, g] @ k[:, g // per].T) * m["scale"]
        if m.get("softcap"):
            s = m["softcap"] * torch.tanh(s / m["softcap"])
        out.append(torch.softmax(s.masked_fill(late, -math.inf), dim=-1) @ v[:, g // per])
    return rounded(torch.stack(out, dim=1))


def attention(h: torch.Tensor, m: dict, w: Dict[str, torch.Tensor], pre: str, eps: float) -> torch.Tensor:
    T, H, G = h.shape[0], m["heads"], m["kv_heads"]
    pos = torch.arange(T)
    q = rounded(rotate_halves(proj(h, w[pre + ".q"]).view(T, H, -1), pos, m.get("rot")))
    k = rounded(rotate_halves(proj(h, w[pre + ".k"]).view(T, G, -1), pos, m.get("rot")))
    v = proj(h, w[pre + ".v"]).view(T, G, -1)
    return proj(causal_softmax(q, k, v, m).reshape(T, -1), w[pre + ".o"])


def keys_as_values_attention(h: torch.Tensor, m: dict, w: Dict[str, torch.Tensor], pre: str, eps: float) -> torch.Tensor:
    """The projected keys are the values; queries and keys then get a norm per head and a rotation, scores a cap, and every
    head's result one gate a token."""
    T, H, G = h.shape[0], m["heads"], m["kv_heads"]
    pos = torch.arange(T)
    q = proj(h, w[pre + ".q"]).view(T, H, -1)
    v = proj(h, w[pre + ".k"]).view(T, G, -1)
    q = rounded(rotate_halves(rms_unit(q, eps) * w[pre + ".q.norm"], pos, m.get("rot")))
    k = rounded(rotate_halves(rms_unit(v, eps) * w[pre + ".k.norm"], pos, m.get("rot")))
    o = causal_softmax(q, k, v, m) * sigmoid(proj(h, w[pre + ".g"]))[:, :, None]
    return proj(o.reshape(T, -1), w[pre + ".o"])


def mlstm_recurrence(q, k, v, i, f):
    """One head's matrix memory, token by token: q, k [T, dim], v [T, dv], log gates i, f [T] -> [T, dv]."""
    T, dk, dv = q.shape[0], q.shape[1], v.shape[1]
    S = torch.zeros(dk, dv, dtype=q.dtype)
    n = torch.zeros(dk, dtype=q.dtype)
    m = torch.zeros((), dtype=q.dtype)
    out = torch.empty(T, dv, dtype=q.dtype)
    for t in range(T):
        m_new = torch.maximum(f[t] + m, i[t])
        keep, put = torch.exp(f[t] + m - m_new), torch.exp(i[t] - m_new)
        S = keep * S + put * torch.outer(k[t], v[t])
        n = keep * n + put * k[t]
        m = m_new
        out[t] = (q[t] @ S) / (torch.maximum((n @ q[t]).abs(), torch.exp(-m)) + 1e-6)
    return out


def mlstm_gates(h: torch.Tensor, m: dict, w: Dict[str, torch.Tensor], pre: str):
    """Log input and forget gates, [T, heads] each."""
    cap = float(m["gate_cap"])
    zi = cap * torch.tanh((proj(h, w[pre + ".i"]) + w[pre + ".i.b"]) / cap)
    zf = cap * torch.tanh((proj(h, w[pre + ".f"]) + w[pre + ".f.b"]) / cap)
    return zi, log_sigmoid(zf)


def mlstm(h: torch.Tensor, m: dict, w: Dict[str, torch.Tensor], pre: str, eps: float) -> torch.Tensor:
    T, H, dk, dv = h.shape[0], m["heads"], m["dim"], m["vdim"]
    q = proj(h, w[pre + ".q"]).view(T, H, dk) * dk ** -0.5
    k = proj(h, w[pre + ".k"]).view(T, H, dk)
    v = proj(h, w[pre + ".v"]).view(T, H, dv)
    i, f = mlstm_gates(h, m, w, pre)
    o = torch.stack([mlstm_recurrence(q[:, g], k[:, g], v[:, g], i[:, g], f[:, g]) for g in range(H)], dim=1)
    y = rms_unit(o, eps).reshape(T, H * dv) * w[pre + ".norm"] * sigmoid(proj(h, w[pre + ".g"]))
    return proj(y, w[pre + ".o"])


MIXERS = {"mlstm": mlstm, "attention": attention, "attention_2": keys_as_values_attention}


# ---- feed-forwards -----------------------------------------------------------------------------------------------------
def dense_ff(h: torch.Tensor, w: Dict[str, torch.Tensor], pre: str) -> torch.Tensor:
    return proj(rounded(gelu_tanh(proj(h, w[pre + ".up"], w[pre + ".up.b"]))), w[pre + ".down"], w[pre + ".down.b"])


def gated_expert(h: torch.Tensor, w: Dict[str, torch.Tensor], pre: str) -> torch.Tensor:
    return proj(rounded(silu(proj(h, w[pre + ".gate"])) * proj(h, w[pre + ".up"])), w[pre + ".down"])


def choose(z: torch.Tensor, correction: torch.Tensor, router: dict) -> torch.Tensor:
    """Router logits of one token [E + identity] -> the chosen experts' numbers, best first."""
    s = torch.softmax(z, dim=-1) + correction
    n, groups = s.numel(), router.get("groups")
    allowed = list(range(n))
    if groups:
        size = n // groups["count"]
        best = sorted(range(groups["count"]), key=lambda g: (-float(s[g * size:(g + 1) * size].max()), g))[:groups["keep"]]
        allowed = [e for e in allowed if e // size in best]
    return torch.tensor(sorted(allowed, key=lambda e: (-float(s[e]), e))[:router["top"]])


def routed_ff(h: torch.Tensor, mlp: dict, w: Dict[str, torch.Tensor], pre: str) -> torch.Tensor:
    r = mlp["router"]
    z = rounded(h) @ w[pre + ".router"].T
    score = torch.softmax(z, dim=-1)
    if _FORCED[0] is not None:
        ids = next(_FORCED[0])
    else:
        ids = torch.stack([choose(z[t], w[pre + ".correction"], r) for t in range(h.shape[0])])
    if _CHOSEN[0] is not None:
        _CHOSEN[0].append(ids)
    y = torch.zeros_like(h)
    for t in range(h.shape[0]):
        chosen = score[t][ids[t]]
        weight = chosen / (chosen.sum() + 1e-20) * r["scale"]
        for e, c in zip(ids[t].tolist(), weight):
            x = h[t:t + 1]
            y[t] += c * (gated_expert(x, w, f"{pre}.e{e}") if e < r["experts"] else rounded(x))[0]
    if mlp.get("shared"):
        y = y + gated_expert(h, w, pre + ".shared") * sigmoid(rounded(h) @ w[pre + ".shared.sg"].T)
    return y


# ---- the model ---------------------------------------------------------------------------------------------------------
def run_order(cfg: dict) -> List[tuple]:
    """(layer, whether a pass begins with it) in the order of the runs."""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return [(i, False) for i in range(n)]
    out = [(i, False) for i in range(loop["start"])]
    for _ in range(loop["times"]):
        out += [(i, i == loop["start"]) for i in range(loop["start"], loop["stop"])]
    return out + [(i, False) for i in range(loop["stop"], n)]


def forward(cfg: dict, w: Dict[str, torch.Tensor], tokens, dtype=torch.float64, round_to=None, forced=None, chosen=None,
            taps: Optional[list] = None) -> torch.Tensor:
    """Logits [T, vocab].  `round_to`: projections' operands and results (and the other tensors an engine keeps in its activations'
    dtype) are rounded to that dtype.  `forced`: per routed feed-forward run, int [T, top], the experts to take whatever the
    scores say; `chosen`: a list that receives what was taken.  `taps`: receives the residual stream after every run."""
    _ROUND[0], _FORCED[0], _CHOSEN[0] = round_to, (iter(forced) if forced is not None else None), chosen
    try:
        w = {k: t.to(dtype) for k, t in w.items()}
        eps = cfg["norm"]["eps"]
        x0 = w["embed"][torch.as_tensor(tokens, dtype=torch.long)]
        x = x0
        for i, begins in run_order(cfg):
            layer = cfg["layers"][i]
            if begins:
                x = rounded(torch.cat([x, x0], dim=-1)) @ w["loop.in"].T
            h = rounded(dynamic_tanh(x, w, f"l{i}.norm1"))
            y = MIXERS[layer["type"]](h, layer["mixer"], w, f"l{i}.mix", eps)
            if layer.get("mlp"):
                y = y + (dense_ff(h, w, f"l{i}.mlp") if layer["mlp"]["kind"] == "dense" else routed_ff(h, layer["mlp"], w, f"l{i}.mlp"))
            x = x + y
            if taps is not None:
                taps.append(x)
        return rounded(dynamic_tanh(x, w, "final.norm")) @ w["head"].T
    finally:
        _ROUND[0] = _FORCED[0] = _CHOSEN[0] = None


def greedy(cfg: dict, w: Dict[str, torch.Tensor], prompt, n: int) -> List[int]:
    """The n tokens greedy decoding appends to `prompt` (the whole sequence is run again for every token)."""
    toks = list(prompt)
    for _ in range(n):
        toks.append(int(torch.argmax(forward(cfg, w, toks)[-1])))
    return toks[len(prompt):]


# ---- configurations and weights for the tests --------------------------------------------------------------------------
def tensor_shapes(cfg: dict) -> Dict[str, tuple]:
    W = cfg["width"]
    out = {"embed": (cfg["vocab"], W), "head": (cfg["vocab"], W)}
    if cfg.get("loop"):
        out["loop.in"] = (W, 2 * W)

    def norm(name):
        out.update({name: (W,), name + ".b": (W,), name + ".alpha": ()})

    norm("final.norm")
    for i, layer in enumerate(cfg["layers"]):
        p, m = f"l{i}", layer["mixer"]
        norm(p + ".norm1")
        if layer["type"] == "mlstm":
            H, dk, dv = m["heads"], m["dim"], m["vdim"]
            out.update({p + ".mix.q": (H * dk, W), p + ".mix.k": (H * dk, W), p + ".mix.v": (H * dv, W), p + ".mix.g": (H * dv, W),
                        p + ".mix.o": (W, H * dv), p + ".mix.norm": (H * dv,), p + ".mix.i": (H, W), p + ".mix.i.b": (H,),
                        p + ".mix.f": (H, W), p + ".mix.f.b": (H,)})
        else:
            H, G, dk, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
            out.update({p + ".mix.q": (H * dk, W), p + ".mix.k": (G * dk, W), p + ".mix.o": (W, H * dv)})
            if layer["type"] == "attention":
                out[p + ".mix.v"] = (G * dv, W)
            else:
                out.update({p + ".mix.g": (H, W), p + ".mix.q.norm": (dk,), p + ".mix.k.norm": (dk,)})
        f = layer.get("mlp")
        if f and f["kind"] == "dense":
            out.update({p + ".mlp.up": (f["ff"], W), p + ".mlp.up.b": (f["ff"],), p + ".mlp.down": (W, f["ff"]), p + ".mlp.down.b": (W,)})
        elif f:
            r = f["router"]
            total = r["experts"] + r.get("identity", 0)
            out.update({p + ".mlp.router": (total, W), p + ".mlp.correction": (total,)})
            parts = [(f".e{e}", f["expert"]["ff"]) for e in range(r["experts"])]
            if f.get("shared"):
                parts.append((".shared", f["shared"]["ff"]))
                out[p + ".mlp.shared.sg"] = (1, W)
            for name, ff in parts:
                out.update({p + ".mlp" + name + ".gate": (ff, W), p + ".mlp" + name + ".up": (ff, W), p + ".mlp" + name + ".down": (W, ff)})
    return out


def random_weights(cfg: dict, seed: int) -> Dict[str, torch.Tensor]:
    """float32 tensors: matrices N(0, 1/in), norm weights near one, biases that spread the forget gates from fast to slow and the
    input gates to both sides of zero, corrections of either sign that change many choices of experts."""
    g = torch.Generator().manual_seed(seed)
    out = {}
    for name, shape in sorted(tensor_shapes(cfg).items()):
        t = torch.randn(shape, generator=g)
        if name.endswith(".alpha"):
            t = 0.6 + 0.1 * t
        elif name.endswith(".mix.f.b"):
            t = 2.5 + 2.0 * t
        elif name.endswith(".mix.i.b"):
            t = -1.0 + 2.0 * t
        elif name.endswith(".b"):
            t = 0.1 * t
        elif name.endswith(".correction"):
            t = 0.15 * t - 0.1
        elif name.endswith(".router"):
            t = 2.0 * t / math.sqrt(shape[1])
        elif len(shape) == 1:
            t = 1.0 + 0.1 * t
        elif name != "embed":
            t = t / math.sqrt(shape[1])
        out[name] = t
    return out


def mlstm_layer(heads, dim, vdim, cap, mlp):
    return {"type": "mlstm", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "gate_cap": cap}, "mlp": mlp}


def attention_layer(kind, heads, kv_heads, dim, vdim, base, dims, mlp, scaling=None, softcap=None, scale=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale if scale is not None else dim ** -0.5,
         "rot": {"base": base, "dims": dims}}
    if scaling:
        m["rot"]["scaling"] = dict(zip(("factor", "original", "fast", "slow"), scaling))
    if softcap:
        m["softcap"] = softcap
    return {"type": kind, "mixer": m, "mlp": mlp}


def dense_mlp(ff):
    return {"kind": "dense", "ff": ff}


def moe_mlp(experts, identity, top, ff, shared_ff=0, groups=None, scale=1.0):
    r = {"experts": experts, "top": top, "scale": scale}
    if identity:
        r["identity"] = identity
    if groups:
        r["groups"] = {"count": groups[0], "keep": groups[1]}
    out = {"kind": "moe", "router": r, "expert": {"ff": ff}}
    if shared_ff:
        out["shared"] = {"ff": shared_ff}
    return out


def config_a():
    """The first two layers run twice (the stream meets itself: x0 beside x0); heads of no multiple of 16 or 8; a part of each
    head turned; more identity experts than others in a group; a layer without a feed-forward."""
    return {"architecture": "Lizezen", "vocab": 61, "width": 40, "norm": {"eps": 1e-5}, "layers": [
        attention_layer("attention", 4, 2, 12, 20, 500.0, 8, moe_mlp(4, 2, 2, 24, 20, (3, 2), 1.7)),
        mlstm_layer(3, 10, 14, 9.0, dense_mlp(70)),
        attention_layer("attention_2", 6, 3, 20, 20, 10000.0, 20, None, scaling=(4.0, 64, 6.0, 1.0), softcap=5.0)],
        "loop": {"start": 0, "stop": 2, "times": 2}}


def config_b():
    """No loop; one group of experts, none of them the identity, no shared expert, one expert a token; scores without a cap where
    the values are the keys and with one where they are not; one key/value head for all, one for each; no rotation in one layer."""
    return {"architecture": "Lizezen", "vocab": 131, "width": 72, "norm": {"eps": 1e-6}, "layers": [
        mlstm_layer(2, 20, 36, 15.0, moe_mlp(5, 0, 1, 40, scale=0.8)),
        attention_layer("attention_2", 3, 1, 24, 24, 1000.0, 16, dense_mlp(96), scaling=(2.5, 100, 8.0, 2.0), scale=0.3),
        attention_layer("attention", 5, 5, 16, 8, 10000.0, 0, None, softcap=8.0),
        mlstm_layer(5, 7, 3, 4.0, None)]}


def config_c():
    """Sizes that take the matrix-core kernels; one layer in the middle runs three times; two groups of which one is kept; top as
    large as a group; heads of 64 and 128 with values of another size."""
    return {"architecture": "Lizezen", "vocab": 300, "width": 128, "norm": {"eps": 1e-5}, "layers": [
        mlstm_layer(2, 64, 128, 12.0, dense_mlp(320)),
        attention_layer("attention_2", 4, 2, 64, 64, 50000.0, 64, moe_mlp(6, 2, 4, 64, 48, (2, 1), 2.0), scaling=(8.0, 512, 16.0, 1.5), softcap=20.0),
        attention_layer("attention", 4, 1, 128, 96, 10000.0, 64, moe_mlp(9, 3, 3, 32, 64, (4, 3), 1.0)),
        mlstm_layer(4, 128, 32, 20.0, dense_mlp(256))],
        "loop": {"start": 1, "stop": 2, "times": 3}}


CONFIGS = {"A": config_a, "B": config_b, "C": config_c}
