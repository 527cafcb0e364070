"""The Moputar design written plainly: one function a mechanism, whole sequences at once, float64 on the CPU.

Nothing here is shared with the engine: the functions take a dict of tensors by checkpoint name and the parsed
config.json, and follow the design's equations directly.  The residual stream is `streams` rows a token, all equal to
the scaled embedding at the start; a sublayer f with its own vectors a, b [streams] and matrix M [streams, streams] does

    u = a X;   y = f(rms(u) * (1 + w));   X' = M^T X + outer(b, y)         (X [streams, width], one token's rows)

with two mixers (a gated delta rule with short convolutions; a softmax attention inside chunks of positions, with short
convolutions, one norm over all of q and one over all of k, rotated pairs, which may read another layer's keys and
values) and a feed-forward down(gelu_tanh(gate h) * up h) that a layer may lack.  The logits come from the rows' sum.
"""
from __future__ import annotations

import math
from typing import Dict, List, Optional

import torch

F64 = torch.float64
_ROUND = None      # a dtype: `forward(..., round_to=)` rounds what an engine in that dtype rounds (see `_r`)


def _r(x: torch.Tensor) -> torch.Tensor:
    """x as it is, or rounded to the dtype a run of `forward` asked for: the rows a projection reads, its result, the normed
    and turned queries and keys, an attention's result.  What the design computes in 32-bit is never rounded."""
    return x if _ROUND is None else x.to(_ROUND).to(F64)


def rms(x: torch.Tensor, eps: float) -> torch.Tensor:
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def silu(x):
    return x * torch.sigmoid(x)


def gelu_tanh(x):
    return 0.5 * x * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (x + 0.044715 * x ** 3)))


def short_conv(u: torch.Tensor, w: torch.Tensor) -> torch.Tensor:
    """u [T, C], w [C, taps]: the last tap takes a token's own row, the one before it the row before; nothing precedes the first."""
    T, C = u.shape
    taps = w.shape[1]
    pad = torch.cat([torch.zeros((taps - 1, C), dtype=u.dtype), u], 0)
    y = torch.zeros_like(u)
    for j in range(taps):
        y = y + pad[j:j + T] * w[:, j]
    return y


def rotate_pairs(x: torch.Tensor, pos: torch.Tensor, rot: Optional[dict]) -> torch.Tensor:
    """x [T, heads, dim]: entries 2i and 2i + 1 turned by pos * base^(-2i/dims), for the first rot.dims entries."""
    if not rot or int(rot["dims"]) == 0:
        return x
    dims = int(rot["dims"])
    f = float(rot["base"]) ** (-2.0 * torch.arange(dims // 2, dtype=F64) / dims)
    ang = pos.to(F64)[:, None] * f[None, :]
    c, s = torch.cos(ang)[:, None, :], torch.sin(ang)[:, None, :]
    out = x.clone()
    u, v = x[..., 0:dims:2], x[..., 1:dims:2]
    out[..., 0:dims:2] = u * c - v * s
    out[..., 1:dims:2] = v * c + u * s
    return out


def visible(T: int, chunk: Optional[int]) -> torch.Tensor:
    i = torch.arange(T)[:, None]
    j = torch.arange(T)[None, :]
    ok = j <= i
    if chunk:
        ok = ok & (i // chunk == j // chunk)
    return ok


def softmax_attention(q, k, v, scale: float, mask: torch.Tensor) -> torch.Tensor:
    """q [T, H, d], k [T, G, d], v [T, G, dv] -> [T, H, dv]; head h reads group h // (H / G)."""
    T, H, _ = q.shape
    per = H // k.shape[1]
    out = torch.zeros((T, H, v.shape[-1]), dtype=q.dtype)
    for h in range(H):
        s = ((q[:, h] @ k[:, h // per].T) * scale).masked_fill(~mask, -math.inf)
        out[:, h] = torch.softmax(s, -1) @ v[:, h // per]
    return out


def attention(W, p: str, mx: dict, h, pos, eps: float, kv=None):
    """Returns (output [T, width], (k, v)); `kv`: another layer's keys and values to read instead of one's own."""
    H, G, dim, vdim = int(mx["heads"]), int(mx["kv_heads"]), int(mx["dim"]), int(mx["vdim"])
    T = h.shape[0]

    def projected(name):
        u = _r(h @ W[p + name].T)
        return short_conv(u, W[p + name + ".conv"]) if mx.get("conv") else u

    def normed(name, heads):
        return _r(rotate_pairs((rms(projected(name), eps) * W[p + name + ".norm"]).view(T, heads, dim), pos, mx.get("rot")))

    q = normed("q", H)
    if kv is None:
        kv = (normed("k", G), _r(projected("v")).view(T, G, vdim))
    mask = visible(T, mx["mask"]["size"] if mx.get("mask") else None)
    o = _r(softmax_attention(q, kv[0], kv[1], float(mx["scale"]), mask))
    return _r(o.reshape(T, H * vdim) @ W[p + "o"].T), kv


def delta_rule(q, k, v, g, beta, S=None):
    """q, k [T, G, dim], v [T, H, vdim], g, beta [T, H] -> (o [T, H, vdim], the last state [H, dim, vdim])."""
    T, H, vdim = v.shape
    per = H // q.shape[1]
    S = torch.zeros((H, q.shape[2], vdim), dtype=q.dtype) if S is None else S.clone()
    qh, kh = q.repeat_interleave(per, 1), k.repeat_interleave(per, 1)
    out = torch.zeros_like(v)
    for t in range(T):
        S = S * g[t][:, None, None]
        u = beta[t][:, None] * (v[t] - torch.einsum("hdv,hd->hv", S, kh[t]))
        S = S + kh[t][:, :, None] * u[:, None, :]
        out[t] = torch.einsum("hdv,hd->hv", S, qh[t])
    return out, S


def delta_mixer(W, p: str, mx: dict, h, eps: float):
    H, G, dim, vdim = int(mx["heads"]), int(mx["kv_heads"]), int(mx["dim"]), int(mx["vdim"])
    T = h.shape[0]
    q, k, v = (silu(short_conv(_r(h @ W[p + n].T), W[p + n + ".conv"])) for n in ("q", "k", "v"))

    def unit(x):
        x = x.view(T, G, dim)
        return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)

    beta = torch.sigmoid(_r(h @ W[p + "b"].T))
    g = torch.exp(-torch.exp(W[p + "A_log"]) * torch.nn.functional.softplus(_r(h @ W[p + "a"].T) + W[p + "dt_bias"]))
    o, _ = delta_rule(unit(q) * dim ** -0.5, unit(k), v.view(T, H, vdim), g, beta)
    o = rms(o, eps) * W[p + "norm"] * silu(_r(h @ W[p + "g"].T)).view(T, H, vdim)
    return _r(_r(o.reshape(T, H * vdim)) @ W[p + "o"].T)


def feed_forward(W, p: str, h):
    return _r(_r(gelu_tanh(_r(h @ W[p + "gate"].T)) * _r(h @ W[p + "up"].T)) @ W[p + "down"].T)


def read_streams(X, a):
    """X [streams, T, width] -> the rows' sum with weights a."""
    return (a[:, None, None] * X).sum(0)


def write_streams(X, M, b, y):
    return torch.stack([sum(M[s, t] * X[s] for s in range(X.shape[0])) + b[t] * y for t in range(X.shape[0])])


def forward(cfg: dict, W: Dict[str, torch.Tensor], tokens: List[int], return_layers: bool = False,
            round_to: Optional[torch.dtype] = None):
    """Logits [T, vocab] of one sequence from its start (and the streams' sum after every layer).  `round_to`: a dtype to which
    the rows a projection reads and what it gives are rounded, as an engine in that dtype does (streams, norms, scores and
    recurrent states stay exact)."""
    global _ROUND
    _ROUND = round_to
    try:
        return _forward(cfg, W, tokens, return_layers)
    finally:
        _ROUND = None


def _forward(cfg, W, tokens, return_layers):
    W = {k: v.to(F64) for k, v in W.items()}
    eps = float(cfg["norm"]["eps"])
    x = W["embed"][torch.tensor(tokens)] * float(cfg.get("embedding", {}).get("scale", 1.0))
    X = x[None].repeat(int(cfg["streams"]), 1, 1)
    pos = torch.arange(len(tokens))
    kvs, layers = {}, []

    def sublayer(X, i, q, f):
        c = f"l{i}.hc{q}."
        y = f(_r(rms(read_streams(X, W[c + "in"]), eps) * (1.0 + W[f"l{i}.norm{q}"])))
        return write_streams(X, W[c + "mix"], W[c + "out"], y)

    for i, ly in enumerate(cfg["layers"]):
        p, mx = f"l{i}.mix.", ly["mixer"]

        def mixer(h):
            if ly["type"] == "delta":
                return delta_mixer(W, p, mx, h, eps)
            src = mx.get("kv_from")
            y, kvs[i] = attention(W, p, mx, h, pos, eps, kvs[src] if src is not None else None)
            return y

        X = sublayer(X, i, 1, mixer)
        if ly.get("mlp"):
            X = sublayer(X, i, 2, lambda h: feed_forward(W, f"l{i}.mlp.", h))
        layers.append(X.sum(0))
    logits = _r(rms(X.sum(0), eps) * (1.0 + W["final.norm"])) @ W["head"].T
    return (logits, torch.stack(layers)) if return_layers else logits


def tensor_shapes(cfg: dict) -> Dict[str, tuple]:
    """Every tensor of a model of this configuration with its shape, as a checkpoint holds them."""
    Wd, n, out = int(cfg["width"]), int(cfg["streams"]), {}
    out["embed"] = (int(cfg["vocab"]), Wd)
    for i, ly in enumerate(cfg["layers"]):
        p, mx = f"l{i}.mix.", ly["mixer"]
        H, G, dim, vdim = int(mx["heads"]), int(mx["kv_heads"]), int(mx["dim"]), int(mx["vdim"])
        for q in (1, 2) if ly.get("mlp") else (1,):
            out[f"l{i}.norm{q}"] = (Wd,)
            out.update({f"l{i}.hc{q}.in": (n,), f"l{i}.hc{q}.out": (n,), f"l{i}.hc{q}.mix": (n, n)})
        if ly["type"] == "delta":
            sizes = {"q": G * dim, "k": G * dim, "v": H * vdim}
            out.update({p + "b": (H, Wd), p + "a": (H, Wd), p + "g": (H * vdim, Wd), p + "A_log": (H,), p + "dt_bias": (H,),
                        p + "norm": (vdim,)})
        else:
            own = mx.get("kv_from") is None
            sizes = {"q": H * dim, "k": G * dim, "v": G * vdim} if own else {"q": H * dim}
            out[p + "q.norm"] = (H * dim,)
            if own:
                out[p + "k.norm"] = (G * dim,)
        for name, rows in sizes.items():
            out[p + name] = (rows, Wd)
            if mx.get("conv"):
                out[p + name + ".conv"] = (rows, int(mx["conv"]))
        out[p + "o"] = (Wd, H * vdim)
        if ly.get("mlp"):
            ff = int(ly["mlp"]["ff"])
            out.update({f"l{i}.mlp.gate": (ff, Wd), f"l{i}.mlp.up": (ff, Wd), f"l{i}.mlp.down": (Wd, ff)})
    out["final.norm"] = (Wd,)
    out["head"] = (int(cfg["vocab"]), Wd)
    return out


# ---- configurations and weights for tests --------------------------------------------------------------------------------
def config_a():
    """Odd sizes, three streams, a reader with wider chunks (and other taps) than its writer."""
    att = {"heads": 4, "kv_heads": 2, "dim": 12, "vdim": 20, "scale": 0.35, "conv": 3, "rot": {"base": 100.0, "dims": 6}}
    return {"architecture": "Moputar", "vocab": 97, "width": 60, "streams": 3, "embedding": {"scale": 2.5}, "norm": {"eps": 1e-5}, "layers": [
        {"type": "attention", "mixer": dict(att, mask={"size": 20}), "mlp": {"kind": "dense", "ff": 44}},
        {"type": "delta", "mixer": {"heads": 6, "kv_heads": 2, "dim": 10, "vdim": 14, "conv": 2}, "mlp": None},
        {"type": "attention", "mixer": dict(att, mask={"size": 33}, kv_from=0, conv=2), "mlp": None},
        {"type": "delta", "mixer": {"heads": 2, "kv_heads": 2, "dim": 24, "vdim": 8, "conv": 5}, "mlp": {"kind": "dense", "ff": 30}}]}


def config_b():
    """One stream, no embedding scale, layers without convolution, mask or rotation, one head, a writer that keeps all keys for
    itself and a reader with chunks."""
    att = {"heads": 3, "kv_heads": 3, "dim": 16, "vdim": 8, "scale": 0.3}
    return {"architecture": "Moputar", "vocab": 130, "width": 96, "streams": 1, "norm": {"eps": 1e-6}, "layers": [
        {"type": "delta", "mixer": {"heads": 1, "kv_heads": 1, "dim": 7, "vdim": 9, "conv": 1}, "mlp": {"kind": "dense", "ff": 72}},
        {"type": "attention", "mixer": dict(att), "mlp": None},
        {"type": "attention", "mixer": dict(att, mask={"size": 50}, kv_from=1), "mlp": {"kind": "dense", "ff": 40}},
        {"type": "attention", "mixer": {"heads": 2, "kv_heads": 1, "dim": 48, "vdim": 48, "scale": 0.2, "rot": {"base": 10000.0, "dims": 48},
                                        "conv": 4}, "mlp": None},
        {"type": "delta", "mixer": {"heads": 3, "kv_heads": 1, "dim": 40, "vdim": 20, "conv": 8}, "mlp": None}]}


def config_c():
    """Sizes the matrix-core kernels take, six streams."""
    att = {"heads": 8, "kv_heads": 2, "dim": 64, "vdim": 64, "scale": 0.15, "conv": 4, "rot": {"base": 5000.0, "dims": 32}}
    return {"architecture": "Moputar", "vocab": 200, "width": 128, "streams": 6, "embedding": {"scale": 8.0}, "norm": {"eps": 1e-5}, "layers": [
        {"type": "delta", "mixer": {"heads": 4, "kv_heads": 2, "dim": 64, "vdim": 32, "conv": 4}, "mlp": {"kind": "dense", "ff": 256}},
        {"type": "attention", "mixer": dict(att, mask={"size": 96}), "mlp": {"kind": "dense", "ff": 128}},
        {"type": "attention", "mixer": dict(att, mask={"size": 40}, kv_from=1), "mlp": None},
        {"type": "delta", "mixer": {"heads": 2, "kv_heads": 1, "dim": 128, "vdim": 128, "conv": 3}, "mlp": None}]}


CONFIGS = {"A": config_a, "B": config_b, "C": config_c}


def random_weights(cfg: dict, seed: int) -> Dict[str, torch.Tensor]:
    """float32 tensors of a size that keeps every mechanism at work: streams that differ, decays spread over (0, 1)."""
    g = torch.Generator().manual_seed(seed)
    out, n = {}, int(cfg["streams"])
    for name, shape in tensor_shapes(cfg).items():
        leaf = name.split(".")[-1]
        r = torch.randn(shape, generator=g)
        if leaf in ("norm1", "norm2") or name == "final.norm":
            t = 0.2 * r
        elif leaf == "norm":
            t = 1.0 + 0.3 * r
        elif leaf == "in":
            t = 1.0 / n + 0.2 * r
        elif leaf == "out":
            t = 1.0 + 0.3 * r
        elif leaf == "mix" and ".hc" in name:
            t = 0.9 * torch.eye(n) + 0.3 * r / math.sqrt(n)
        elif leaf == "A_log":
            t = torch.log(0.05 + 1.5 * torch.rand(shape, generator=g))
        elif leaf == "dt_bias":
            t = -2.5 + r
        elif leaf == "conv":
            t = 0.6 * r
        elif name == "embed":
            t = r / float(cfg.get("embedding", {}).get("scale", 1.0))
        elif len(shape) == 2:
            t = r * (1.3 / math.sqrt(shape[1]))
        else:
            t = r
        out[name] = t
    return out
