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
