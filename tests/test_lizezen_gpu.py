"""The Lizezen design in the engine against the plain implementation (`plain_lizezen.py`): the new kernels alone, every mechanism
alone in a one-layer model (with a key made to stand out far back and at page borders, gates that make the denominator's floor and the
running maximum count), then whole models through the engine's own step function (whole prompts, decoding token by token, portions
down to two tokens, mixed batches with pages and slots used again, recorded steps) and through the entry point with its scheduler
(greedy generation).  Configurations A, B and C differ in every size and switch (see plain_lizezen)."""
import json
import math
import os

import pytest
import torch

import plain_lizezen as P
from helpers import TOL, Driver, rel_err

pytestmark = pytest.mark.gpu
DEV = "cuda:0"
BF, F32, F64 = torch.bfloat16, torch.float32, torch.float64


@pytest.fixture(scope="module")
def K():
    from infinilm_amd import kernels
    return kernels


def make_dir(path, cfg, W, store):
    from safetensors.torch import save_file
    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as fh:
        json.dump(cfg, fh)
    save_file({k: v.to(getattr(torch, store)).contiguous() for k, v in W.items()}, os.path.join(path, "model.safetensors"))
    return {k: v.to(getattr(torch, store)).to(torch.float32) for k, v in W.items()}


def tokens(cfg, n, seed):
    g = torch.Generator().manual_seed(seed)
    return torch.randint(0, cfg["vocab"], (n,), generator=g).tolist()


def _close(got, want, tol, what):
    err = rel_err(got, want)
    assert err < tol, f"{what}: error {err:.3e}"


def i32(*v):
    return torch.tensor(v, dtype=torch.int32, device=DEV)


# ---- the kernels alone ------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("H,T,dtype", [(64, 5, "float32"), (61, 3, "float32"), (4096, 70, "bfloat16"), (1028, 2, "bfloat16"), (50, 9, "bfloat16"), (6, 1, "float32")])
def test_dynamic_tanh_and_rows_beside(K, H, T, dtype):
    """Sums of no, one and six addends of every kind (bfloat16 rows, float parts, one row for all) and both results."""
    dt = getattr(torch, dtype)
    g = torch.Generator().manual_seed(H)
    r, x0 = torch.randn((T, H), generator=g), torch.randn((T, H), generator=g)
    w, b, alpha = torch.randn((H,), generator=g).to(dt), torch.randn((H,), generator=g).to(dt), torch.tensor(0.37)
    rows, parts, one = torch.randn((T, H), generator=g).to(BF), torch.randn((3, T, H), generator=g), torch.randn((H,), generator=g).to(dt)
    kinds = [(rows, 0.5), (parts, 1.0), (one, -2.0), (x0, 1.0), (one, 1.0), (parts, 0.25)]
    for n in (0, 1, 6):
        want = r.double()
        for a, s in kinds[:n]:
            want = want + s * (a.double().sum(0) if a.dim() == 3 else a.double())
        add = [(a.to(DEV), s) for a, s in kinds[:n]]
        stream = r.to(DEV).clone()
        y = K.add_dynamic_tanh(stream, add, alpha.to(DEV), w.to(DEV), b.to(DEV), dt)
        tol = 2e-6 if dt == F32 else 6e-3
        _close(y, torch.tanh(0.37 * want) * w.double() + b.double(), tol, f"{n} addends")
        _close(stream, want, 2e-6, "the stream itself")
        _close(K.add_dynamic_tanh(r.to(DEV).clone(), add, alpha.to(DEV), w.to(DEV), None, dt), torch.tanh(0.37 * want) * w.double(), tol, "no bias")
        stream = r.to(DEV).clone()
        y = K.add_beside(stream, add, x0.to(DEV), dt)
        _close(y, torch.cat([want, x0.double()], dim=1), tol, "rows beside")
        _close(stream, want, 2e-6, "the stream beside")


def _turned(x, pos, freq, mag, rd):
    """Pairs (i, i + rd / 2) turned by the float32 angle."""
    n = rd // 2
    ang = (pos.to(F32)[:, None] * freq[None]).double()
    c, s = (torch.cos(ang) * mag)[:, None], (torch.sin(ang) * mag)[:, None]
    out = x.clone()
    out[..., :n], out[..., n:rd] = x[..., :n] * c - x[..., n:rd] * s, x[..., n:rd] * c + x[..., :n] * s
    return out


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("nh,nkv,d,dn,dv,rd,mag,keys,norm,page", [(4, 2, 64, 64, 64, 64, 1.0, False, False, 16), (6, 3, 32, 20, 20, 20, 1.14, True, True, 4),
                                                                 (8, 2, 128, 128, 128, 64, 1.2, True, True, 64), (3, 1, 96, 96, 48, 96, 1.0, False, True, 64),
                                                                 (5, 5, 48, 48, 48, 32, 1.3, True, False, 16), (4, 4, 16, 7, 16, 6, 1.0, False, True, 16),
                                                                 (2, 1, 256, 256, 256, 0, 1.0, True, True, 32), (33, 1, 80, 80, 80, 16, 0.9, True, True, 16)])
def test_keys_as_values_and_half_pairs(K, nh, nkv, d, dn, dv, rd, mag, keys, norm, page, dtype):
    """Norm, turn and cache write of both kernels (wide pieces and any size) at far positions; the values in the cache are the keys
    before norm and turn; gate columns behind the rows are left alone."""
    dt = getattr(torch, dtype)
    g = torch.Generator().manual_seed(nh * d + rd)
    T, pages = 19, -(-19 // page) + 1
    heads = nh + (1 if keys else 2) * nkv
    x = torch.randn((T, heads, d), generator=g).to(dt)
    x[:, :nh + nkv, dn:] = 0
    if not keys:
        x[:, nh + nkv:, dv:] = 0
    rows = torch.zeros((T, -(-(heads * d + nh) // 8) * 8), dtype=dt)
    rows[:, :heads * d] = x.reshape(T, -1)
    rows[:, heads * d:] = 5.0
    pos = torch.randint(0, 5000, (T,), generator=g, dtype=torch.int32)
    freq = torch.rand((max(rd // 2, 1),), generator=g)[:rd // 2]
    wq, wk = ((1 + 0.2 * torch.randn((dn,), generator=g)).to(dt) for _ in range(2)) if norm else (None, None)
    perm = torch.randperm(pages * page, generator=g)[:T].to(torch.int32)
    kc, vc = torch.zeros((pages, nkv, page, d), dtype=dt, device=DEV), torch.zeros((pages, nkv, d, page), dtype=dt, device=DEV)
    dr = rows.to(DEV)
    K.qkv_norm_rope_kvwrite(dr[:, :heads * d], pos.to(DEV), freq.to(DEV) if rd else None, wq.to(DEV) if norm else None, wk.to(DEV) if norm else None,
                            kc, vc, perm.to(DEV), nh, nkv, d, dn, dv, rd, False, 1e-5, half=True, magnitude=mag, values_are_keys=keys)
    q, k = x[:, :nh, :dn].double(), x[:, nh:nh + nkv, :dn].double()
    v = x[:, nh:nh + nkv] if keys else x[:, nh + nkv:]
    if norm:
        q, k = P.rms_unit(q, 1e-5) * wq.double(), P.rms_unit(k, 1e-5) * wk.double()
    if rd:
        q, k = _turned(q, pos, freq, mag, rd), _turned(k, pos, freq, mag, rd)
    tol = 4e-6 if dt == F32 else 6e-3
    out = dr.cpu()
    _close(out[:, :nh * d].view(T, nh, d)[..., :dn], q, tol, "queries")
    assert (out[:, :nh * d].view(T, nh, d)[..., dn:] == 0).all() and (out[:, heads * d:] == 5.0).all()
    at = perm.long()
    got_k = torch.stack([kc.cpu()[s // page, :, s % page] for s in at])
    got_v = torch.stack([vc.cpu()[s // page, :, :, s % page] for s in at])
    _close(got_k[..., :dn], k, tol, "keys in the cache")
    assert torch.equal(got_v[..., :dv], v[..., :dv]) and (got_k[..., dn:] == 0).all()


def test_head_gate(K):
    g = torch.Generator().manual_seed(2)
    for T, H, d, dt in ((5, 3, 20, F32), (70, 8, 128, BF), (2, 5, 48, BF), (3, 1, 7, F32)):
        o, rows = torch.randn((T, H * d), generator=g).to(dt), 3 * torch.randn((T, H + 6), generator=g).to(dt)
        want = (o.double().view(T, H, d) * P.sigmoid(rows[:, 2:2 + H].double())[..., None]).reshape(T, -1)
        got = K.head_gate_(o.to(DEV), rows.to(DEV)[:, 2:2 + H], H, d)
        _close(got, want, 2e-6 if dt == F32 else 6e-3, f"{T} x {H} x {d}")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("kind", ["gelu_tanh", "relu2", "silu"])
def test_product_with_bias_and_activation(K, kind, dtype):
    """Every row count at which the kernel changes, with and without a bias, few and many outputs."""
    dt = getattr(torch, dtype)
    act = {"gelu_tanh": P.gelu_tanh, "relu2": lambda z: torch.clamp(z, min=0) ** 2, "silu": P.silu}[kind]
    g = torch.Generator().manual_seed(4)
    for N, Kd in ((72, 40), (8200, 64), (8320, 264)):
        w, b = (torch.randn((N, Kd), generator=g) / math.sqrt(Kd)).to(dt), torch.randn((N,), generator=g).to(dt)
        x = torch.randn((210, Kd), generator=g).to(dt)
        for M in (1, 16, 17, 32, 33, 64, 65, 112, 113, 210):
            for bias in (b, None):
                z = x[:M].double() @ w.double().T + (0 if bias is None else bias.double())
                got = K.linear_activation(x[:M].to(DEV), w.to(DEV), None if bias is None else bias.to(DEV), kind)
                _close(got, act(z), 4e-6 if dt == F32 else 1.2e-2, f"{M} x {N} x {Kd}, bias {bias is not None}")
            _close(K.gemm(x[:M].to(DEV), w.to(DEV), b.to(DEV)), x[:M].double() @ w.double().T + b.double(), 4e-6 if dt == F32 else 8e-3, f"product {M} x {N}")


@pytest.mark.parametrize("E,ident,groups,keep,top,T", [(4, 2, 3, 2, 2, 50), (13, 3, 4, 2, 3, 33), (5, 0, 1, 1, 1, 7), (6, 2, 2, 1, 4, 300), (1, 1, 1, 1, 2, 5),
                                                       (100, 28, 8, 2, 9, 65), (300, 20, 64, 5, 8, 20), (3, 9, 4, 4, 3, 129), (700, 68, 256, 90, 16, 9)])
def test_routing_by_groups(K, E, ident, groups, keep, top, T):
    """Corrections of either sign (choice scores below zero included), groups, identity experts, weights divided by their sum; the
    pairs' order holds exactly those of experts with matrices."""
    g = torch.Generator().manual_seed(E + top)
    n = E + ident
    z, corr = 2 * torch.randn((T, n + 1), generator=g), 0.4 * torch.randn((n,), generator=g) - 0.3
    plan = K.moe_route(z.to(DEV), E, top, softmax=True, weight_scale=1.7, identity=ident, correction=corr.to(DEV), groups=groups, keep=keep, normalise=True)
    router = {"top": top, "groups": {"count": groups, "keep": keep}}
    s = torch.softmax(z[:, :n].double(), -1)
    ids, wts, inv = plan.ids.cpu().long(), plan.weights.cpu(), plan.inv.cpu().view(T, top)
    for t in range(T):
        assert ids[t].tolist() == P.choose(z[t, :n].double(), corr.double(), router).tolist(), t
    chosen = s.gather(1, ids)
    _close(wts, chosen / (chosen.sum(-1, keepdim=True) + 1e-20) * 1.7, 2e-6, "weights")
    real = ids < E
    assert (inv[~real] == -1).all() and sorted(inv[real].tolist()) == list(range(int(real.sum())))
    perm, off = plan.perm.cpu().long(), plan.offsets.cpu().long()
    assert int(off[E]) == int(real.sum())
    for e in range(E):
        assert all(int(ids.view(-1)[p]) == e for p in perm[off[e]:off[e + 1]])


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("W,ff,shared,T", [(40, 24, 20, 5), (64, 32, 0, 130), (128, 64, 96, 1), (128, 64, 96, 900), (50, 30, 17, 40)])
def test_experts_alone(W, ff, shared, T, dtype):
    """The whole feed-forward (products in both tile sizes, sums over chosen experts, identity experts, the shared expert and its
    number) against the plain one that is made to choose alike."""
    from infinilm_amd.parts import BuildContext
    from infinilm_amd.parts.moe import RoutedGatedExperts
    dt = getattr(torch, dtype)
    mlp = P.moe_mlp(5, 3, 3, ff, shared, (4, 3), 2.5)
    cfg = {"architecture": "Lizezen", "vocab": 3, "width": W, "norm": {"eps": 1e-5}, "layers": [P.mlstm_layer(1, 4, 4, 5.0, mlp)]}
    w = {k[len("l0.mlp."):]: t.to(dt) for k, t in P.random_weights(cfg, W + T).items() if k.startswith("l0.mlp.")}
    part = RoutedGatedExperts(W, 5, 3, ff, BuildContext(dtype=dt, device=torch.device(DEV)), identity=3, groups=4, keep=3, weight_scale=2.5, shared_ff=shared)
    named = part.named_parameters()
    assert set(named) == set(w)
    for k, p in named.items():
        p.store(w[k])
    g = torch.Generator().manual_seed(T)
    h = torch.randn((T, W), generator=g).to(dt)
    RoutedGatedExperts.trace = []
    try:
        y = part.forward(h.to(DEV), None)
        ids = RoutedGatedExperts.trace[0].cpu().long()
    finally:
        RoutedGatedExperts.trace = None
    P._FORCED[0] = iter([ids])
    try:
        want = P.routed_ff(h.double(), mlp, {"m." + k: t.double() for k, t in w.items()}, "m")
    finally:
        P._FORCED[0] = None
    free = [P.choose(z, w["correction"].double(), mlp["router"]).tolist() for z in h.double() @ w["router"].double().T]
    agree = sum(sorted(a) == sorted(b) for a, b in zip(free, ids.tolist())) / T
    assert agree == 1.0 if dt == F32 else agree > 0.97
    _close(y, want, 6e-6 if dt == F32 else 1.5e-2, "experts")


# ---- the recurrence alone ----------------------------------------------------------------------------------------------
def _mlstm_case(K, H, dk, dv, seqs, cuts, rows_dt, out_dt, shift_i=0.0, shift_f=3.0, cap=15.0, seed=0, slots=None):
    """`seqs` sequences of rows through launches that take `cuts[launch][sequence]` tokens of each (0: absent), states in pool rows
    that are permuted; results per sequence beside the plain recurrence's."""
    g = torch.Generator().manual_seed(seed + H * dk + dv)
    ip = -(-(H * (2 * dk + 2 * dv) + H) // 8) * 8
    width = -(-(ip + H) // 8) * 8
    i_off, f_off, g_off = H * (2 * dk + 2 * dv), ip, H * (2 * dk + dv)
    u = [torch.randn((n, width), generator=g) for n in seqs]
    for x in u:
        x[:, i_off:] *= 3.0
    u = [x.to(rows_dt) for x in u]
    bi, bf = torch.randn((H,), generator=g) + shift_i, torch.randn((H,), generator=g) + shift_f
    w = (1 + 0.2 * torch.randn((H * dv,), generator=g)).to(out_dt)
    R = len(seqs)
    rows = [1 + p for p in torch.randperm(R + 1, generator=g)[:R].tolist()]
    pool, pm = torch.full((R + 3, H, dv + 1, dk), 9.0, device=DEV), torch.full((R + 3, H), 9.0, device=DEV)
    pool[0], pm[0] = 0, 0
    at, got = [0] * R, [[] for _ in range(R)]
    for cut in cuts:
        live = [r for r in range(R) if cut[r]]
        x = torch.cat([u[r][at[r]:at[r] + cut[r]] for r in live]).to(DEV)
        off = [0]
        for r in live:
            off.append(off[-1] + cut[r])
        y = K.mlstm(x, bi.to(DEV), bf.to(DEV), i_off, f_off, g_off, H, dk, dv, cap, pool, pm, i32(*[rows[r] if at[r] else 0 for r in live]),
                    i32(*[rows[r] for r in live]), i32(*off), len(live), w.to(DEV), 1e-5, out_dt, max_len=max(cut))
        for j, r in enumerate(live):
            got[r].append(y[off[j]:off[j + 1]].cpu())
            at[r] += cut[r]
    assert at == list(seqs) and (pool[0] == 0).all() and (pm[0] == 0).all()
    want = []
    for x in u:
        x = x.double()
        n = x.shape[0]
        q, k = x[:, :H * dk].view(n, H, dk) * dk ** -0.5, x[:, H * dk:2 * H * dk].view(n, H, dk)
        v, gate = x[:, 2 * H * dk:g_off].view(n, H, dv), x[:, g_off:g_off + H * dv]
        li = cap * torch.tanh((x[:, i_off:i_off + H] + bi.double()) / cap)
        lf = P.log_sigmoid(cap * torch.tanh((x[:, f_off:f_off + H] + bf.double()) / cap))
        o = torch.stack([P.mlstm_recurrence(q[:, h], k[:, h], v[:, h], li[:, h], lf[:, h]) for h in range(H)], 1)
        want.append(P.rms_unit(o, 1e-5).reshape(n, -1) * w.double() * P.sigmoid(gate))
    return [torch.cat(x) for x in got], want


SIZES = [(3, 48, 80), (2, 128, 128), (3, 10, 14), (1, 7, 3), (2, 64, 200), (5, 16, 16), (2, 200, 24), (1, 256, 140), (2, 300, 20), (2, 33, 100), (1, 4, 1000)]


@pytest.mark.parametrize("rows", ["float32", "bfloat16"])
@pytest.mark.parametrize("H,dk,dv", SIZES)
def test_mlstm_recurrence(K, H, dk, dv, rows):
    """Segments on either side of the chunked form's length in one launch, portions of two tokens and single tokens after long ones,
    states carried from launch to launch in rows that held something else; every block shape of the step kernel, both chunked
    forms and the sizes beyond them.  Results in float show that bfloat16 rows lose nothing on the way."""
    seqs = [200, 37, 3, 131]
    cuts = [(130, 1, 0, 31), (2, 33, 1, 32), (1, 2, 1, 65), (66, 0, 1, 2), (1, 1, 0, 1)]
    got, want = _mlstm_case(K, H, dk, dv, seqs, cuts, getattr(torch, rows), F32)
    for r, (a, b) in enumerate(zip(got, want)):
        _close(a, b, 3e-5, f"sequence {r}")
    if rows == "bfloat16":
        got, want = _mlstm_case(K, H, dk, dv, [90, 2], [(64, 1), (26, 1)], BF, BF)
        for a, b in zip(got, want):
            _close(a, b, 1e-2, "bfloat16 results")


@pytest.mark.parametrize("rows", ["float32", "bfloat16"])
@pytest.mark.parametrize("shift_i,shift_f,cap", [(-30.0, 20.0, 12.0), (40.0, 20.0, 30.0), (0.0, -40.0, 15.0), (0.0, 40.0, 15.0), (-10.0, -10.0, 4.0), (5.0, 0.0, 80.0)])
def test_mlstm_gates_at_their_ends(K, shift_i, shift_f, cap, rows):
    """Input gates far below zero (the denominator's floor and the start at a maximum of zero count), far above; everything
    forgotten at once, and nothing at all; a cap that bites and one that never does."""
    got, want = _mlstm_case(K, 2, 24, 40, [300, 60], [(200, 1), (98, 40), (1, 19), (1, 0)], getattr(torch, rows), F32, shift_i, shift_f, cap, seed=7)
    for a, b in zip(got, want):
        _close(a, b, 5e-5, "gates at their ends")


def test_mlstm_pieces(K):
    """Every piece length gives the same result up to rounding (long segments in one and in many pieces)."""
    old = K.MLSTM_PIECE
    try:
        for rows in (F32, BF):
            ref = None
            for piece in (64, 128, 192, 1024):
                K.MLSTM_PIECE = piece
                got, want = _mlstm_case(K, 2, 40, 48, [700, 70, 190], [(700, 70, 129), (0, 0, 61)], rows, F32, seed=3)
                for r, (a, b) in enumerate(zip(got, want)):
                    _close(a, b, 3e-5, f"pieces of {piece}, sequence {r}")
                if ref is not None:
                    _close(got[0], ref, 2e-5, "piece lengths")
                ref = got[0]
    finally:
        K.MLSTM_PIECE = old


# ---- one mechanism in a one-layer model ---------------------------------------------------------------------------------
def _one_layer(layer, width=48):
    return {"architecture": "Lizezen", "vocab": 50, "width": width, "norm": {"eps": 1e-5}, "layers": [layer]}


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("kind,dim,vdim,page,dims", [("attention", 64, 48, 64, 16), ("attention", 12, 20, 4, 4), ("attention", 128, 128, 16, 32),
                                                     ("attention_2", 64, 64, 64, 8), ("attention_2", 20, 20, 16, 4), ("attention_2", 128, 128, 32, 16)])
def test_a_far_key(kind, dim, vdim, page, dims, dtype, tmp_path):
    """A token whose key outweighs all others for every query (its own embedding row makes it so), at a sequence's start, on both
    sides of a page border and in the middle: in a prompt, in portions and for decoded tokens hundreds of positions later.  Where
    the values are the keys before norm and turn, what shows is that row."""
    layer = P.attention_layer(kind, 4, 2, dim, vdim, 1e5, dims, None, scaling=(4.0, 64, 6.0, 1.0) if kind == "attention_2" else None,
                              softcap=60.0 if kind == "attention_2" else None, scale=3.0 / math.sqrt(dim))
    cfg = _one_layer(layer)
    W = P.random_weights(cfg, 5)
    g = torch.Generator().manual_seed(1)
    loud, all_dir, dirs = (torch.randn((n,), generator=g) for n in (48, 48, dim))
    dirs[:dims] = 0                                   # (the turned entries stay out of it: the score does not depend on the distance)
    W["embed"] = 0.3 * W["embed"] + all_dir           # every token's query holds `dirs`
    W["embed"][7] = 4.0 * loud                         # token 7's key does, and strongly
    W["l0.norm1"].fill_(1.0)
    W["l0.norm1.alpha"].fill_(0.3)
    W["l0.mix.q"] += (dirs.repeat(4)[:, None] * all_dir[None] / all_dir.norm() ** 2) * 3
    W["l0.mix.k"] += (dirs.repeat(2)[:, None] * loud[None] / loud.norm() ** 2) * 3
    base = [t if t != 7 else 8 for t in tokens(cfg, 280, 3)]
    d = str(tmp_path / "m")
    Wr = make_dir(d, cfg, W, dtype)
    drv = Driver(d, dtype, num_pages=-(-280 // page) + 1, page_size=page, max_requests=2)
    quiet = P.forward(cfg, Wr, base)
    for i, at in enumerate((0, 1, 63, 64, 130)):
        toks = list(base)
        toks[at] = 7
        want = P.forward(cfg, Wr, toks)
        assert rel_err(want[at + 1:], quiet[at + 1:]) > 0.05, "the marked key does not show"
        assert rel_err(want[250:], quiet[250:]) > 0.03, "the marked key does not show far on"
        rid = f"r{i}"
        cuts = [(280,), (150, 2, 50) + (1,) * 78, (247,) + (1,) * 33][i % 3]
        a = 0
        for n in cuts:
            drv.step([(rid, toks[a:a + n])], end=[rid] if a + n == 280 else [])
            a += n
        _close(drv.request_logits(rid, 280), want, TOL[dtype], f"marked key at {at}")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("dim,vdim", [(10, 14), (64, 64), (128, 128), (160, 40)])
def test_the_memory_lasts_through_portions(dim, vdim, dtype, tmp_path):
    """Forget gates near one: a token 290 positions back still shows, through portions on either side of the chunks' length and
    decoded tokens; with input gates of one token far above all others its content stands out."""
    cfg = _one_layer(P.mlstm_layer(2, dim, vdim, 15.0, None))
    W = P.random_weights(cfg, 9)
    W["l0.mix.f.b"].fill_(12.0)
    loud = torch.randn((48,), generator=torch.Generator().manual_seed(3))
    W["embed"][7] = 3.0 * loud
    W["l0.mix.i"] += 8.0 * loud[None] / loud.norm() ** 2
    toks = [t if t != 7 else 8 for t in tokens(cfg, 320, 4)]
    toks[30] = 7
    d = str(tmp_path / "m")
    Wr = make_dir(d, cfg, W, dtype)
    want = P.forward(cfg, Wr, toks)
    other = list(toks)
    other[30] = 8
    assert rel_err(P.forward(cfg, Wr, other)[-1], want[-1]) > 0.02
    drv = Driver(d, dtype, num_pages=1, page_size=16, max_requests=2)
    at = 0
    for n in [2, 131, 3, 64, 31, 33, 30]:
        drv.step([("a", toks[at:at + n])])
        at += n
    for i in range(at, 320):
        drv.step([("a", [toks[i]])])
    got = drv.request_logits("a", 320)
    bound = TOL[dtype] if dtype == "float32" else max(TOL[dtype], 2 * rel_err(P.forward(cfg, Wr, toks, round_to=BF), want))
    _close(got, want, bound, "memory through portions")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_first_tokens_of_a_sequence(dtype, tmp_path):
    """The first tokens (an empty memory whose maximum starts at zero: input gates far below it let the floor of the denominator
    show; one key), alone, in twos and whole, in slots and pages another request has used."""
    cfg = P.config_a()
    W = P.random_weights(cfg, 2)
    W["l1.mix.i.b"].fill_(-6.0)
    d = str(tmp_path / "m")
    W = make_dir(d, cfg, W, dtype)
    drv = RoutedDriver(d, dtype, num_pages=6, page_size=16, max_requests=1)
    drv.step([("x", tokens(cfg, 40, 9))], end=["x"])
    for i, cut in enumerate(((1,) * 6, (2, 2, 2), (6,), (1, 5), (3, 1, 2))):
        toks, a = tokens(cfg, 6, 20 + i), 0
        for n in cut:
            drv.step([(f"r{i}", toks[a:a + n])], end=[f"r{i}"] if a + n == 6 else [])
            a += n
        _compare(cfg, W, toks, drv, f"r{i}", dtype, f"cut {cut}")


def test_the_stream_after_every_run(tmp_path):
    """The dump of the residual stream after every run of a looped model (before what comes ahead of the next pass)."""
    from infinilm_amd.engine.loading import load_model, make_runner
    from infinilm_amd.engine.step import StepEntry
    for name in ("A", "C"):
        cfg = P.CONFIGS[name]()
        d = str(tmp_path / name)
        W = make_dir(d, cfg, P.random_weights(cfg, 6), "float32")
        runner = make_runner(load_model(d, "float32", DEV), num_pages=8, page_size=16, max_requests=2)
        toks, layers, taps = tokens(cfg, 30, 1), [], {}
        logits = P.forward(cfg, W, toks, taps=layers)
        runner.cache.admit("a")
        got = runner.step([StepEntry("a", toks, [3, 29])], taps=taps)
        _close(got, logits[[3, 29]], TOL["float32"], "logits")
        for i, want in enumerate(layers):
            residual, pending, scale = taps[f"run{i}"]
            x = residual.double().cpu()
            if pending is not None:
                x = x + scale * (pending.double().sum(0) if pending.dim() == 3 else pending.double()).cpu()
            _close(x, want, TOL["float32"], f"stream after run {i}")


# ---- whole models through the step function -----------------------------------------------------------------------------
class RoutedDriver(Driver):
    """The helper's driver, which also files the experts the engine chose under (request, position)."""

    def __init__(self, *a, **k):
        super().__init__(*a, **k)
        self.picks = {}

    def step(self, entries, want_all=True, end=()):
        from infinilm_amd.parts.moe import RoutedGatedExperts
        starts = [self.runner.cache.length(rid) if self.runner.cache.has(rid) else 0 for rid, _ in entries]
        RoutedGatedExperts.trace = []
        try:
            super().step(entries, want_all=want_all, end=end)
            calls = [t.cpu().long() for t in RoutedGatedExperts.trace]
        finally:
            RoutedGatedExperts.trace = None
        row = 0
        for (rid, toks), s in zip(entries, starts):
            for i in range(len(toks)):
                self.picks[(rid, s + i)] = [c[row] for c in calls]
                row += 1

    def request_picks(self, rid, n):
        runs = len(self.picks[(rid, 0)])
        return [torch.stack([self.picks[(rid, i)][r] for i in range(n)]) for r in range(runs)]


def _compare(cfg, W, toks, drv, rid, dtype, what):
    """float32: every logit and every choice of experts as the plain implementation's.  bfloat16: the choices may differ where the
    plain scores are close; the logits follow the plain implementation run with the engine's choices.  A head's result divided by
    its own root mean square multiplies a rounding error many times at the few positions where that happens to be small, in the
    plain implementation with rounded projections too, at positions of its own: most positions (the median) are held closely to
    what that one loses, the worst loosely."""
    n = len(toks)
    got, picks = drv.request_logits(rid, n).double(), drv.request_picks(rid, n)
    if dtype == "float32":
        free = []
        want = P.forward(cfg, W, toks, chosen=free)
        for a, b in zip(free, picks):
            assert torch.equal(a.sort(-1).values, b.sort(-1).values), f"{what}: other experts"
        err = rel_err(got, want)
        print(f"[err] {what} {dtype} n={n}: {err:.3e}")
        assert err < TOL[dtype], f"{what} {dtype}: error {err:.3e}"
        return
    want = P.forward(cfg, W, toks, forced=picks)
    top = max(1.0, float(want.abs().max()))
    e = (got - want).abs().amax(-1) / top
    l = (P.forward(cfg, W, toks, forced=picks, round_to=BF) - want).abs().amax(-1) / top
    what = f"{what} {dtype}: median {float(e.median()):.3e} (plain, rounded: {float(l.median()):.3e}), worst {float(e.max()):.3e} ({float(l.max()):.3e})"
    print(f"[err] {what} n={n}")
    assert float(e.median()) < max(TOL["bfloat16"] / 4, 2.0 * float(l.median())), what
    assert float(e.max()) < max(TOL["bfloat16"], 4.0 * float(l.max())), what


CASES = [(c, d, p) for d in ("float32", "bfloat16") for c, p in (("A", 16), ("B", 64), ("C", 64), ("C", 32), ("A", 4))]


@pytest.fixture(scope="module", params=CASES, ids=[f"{c}-{d}-p{p}" for c, d, p in CASES])
def case(request, tmp_path_factory):
    name, dtype, page = request.param
    cfg = P.CONFIGS[name]()
    d = tmp_path_factory.mktemp(f"lizezen_{name}_{dtype}")
    W = make_dir(str(d), cfg, P.random_weights(cfg, 40 + ord(name)), dtype)
    toks = {r: tokens(cfg, n, 11 * i + 3) for i, (r, n) in
            enumerate([("r0", 230), ("r1", 1), ("r2", 45), ("r3", 70), ("r4", 2), ("r5", 131)])}
    return {"cfg": cfg, "dir": str(d), "dtype": dtype, "toks": toks, "name": name, "page": page, "W": W}


def _check(case, drv, rid):
    _compare(case["cfg"], case["W"], case["toks"][rid], drv, rid, case["dtype"], f"{case['name']} {rid}")


def _pages(n, page):
    return -(-n // page)


def test_whole_requests(case):
    page = case["page"]
    drv = RoutedDriver(case["dir"], case["dtype"], num_pages=_pages(230, page) + 1, page_size=page, max_requests=2)
    for rid, t in case["toks"].items():
        drv.step([(rid, t)], end=[rid])
        _check(case, drv, rid)


def test_last_tokens_one_by_one(case):
    """The last 90 tokens decoded one by one (over page borders)."""
    page = case["page"]
    drv = RoutedDriver(case["dir"], case["dtype"], num_pages=_pages(230, page) + 1, page_size=page, max_requests=2)
    for rid in ("r0", "r1", "r4", "r5"):
        t = case["toks"][rid]
        head = max(len(t) - 90, 0)
        if head:
            drv.step([(rid, t[:head])])
        for i in range(head, len(t)):
            drv.step([(rid, [t[i]])], end=[rid] if i == len(t) - 1 else [])
        _check(case, drv, rid)


def test_portions_of_changing_size(case):
    page = case["page"]
    drv = RoutedDriver(case["dir"], case["dtype"], num_pages=_pages(230, page) + 1, page_size=page, max_requests=2)
    sizes = [2, 5, page, 3, 2 * page + 1, 2, 17, page - 1, 1, 64]
    for rid in ("r0", "r2", "r5"):
        t = case["toks"][rid]
        at, i = 0, 0
        while at < len(t):
            n = max(1, min(sizes[i % len(sizes)], len(t) - at))
            drv.step([(rid, t[at:at + n])], end=[rid] if at + n == len(t) else [])
            at, i = at + n, i + 1
        _check(case, drv, rid)


def test_mixed_steps_reuse_pages_and_slots(case):
    """Four request slots and pages for about two long requests serve six requests: portions of some beside single tokens of
    others; a request that ends frees its slot and pages for the next."""
    page, toks = case["page"], case["toks"]
    drv = RoutedDriver(case["dir"], case["dtype"], num_pages=_pages(230, page) + _pages(131, page) + _pages(70, page) + 3, page_size=page, max_requests=4)
    at = {r: 0 for r in toks}

    def take(rid, n):
        a = at[rid]
        at[rid] = min(a + n, len(toks[rid]))
        return (rid, toks[rid][a:at[rid]])

    def run(plan):
        entries = [take(r, n) for r, n in plan if at[r] < len(toks[r])]
        if entries:
            drv.step(entries, end=[r for r, _ in entries if at[r] == len(toks[r])])

    run([("r1", 1), ("r0", 70), ("r2", 3)])
    run([("r0", 2), ("r2", 40), ("r4", 1)])
    run([("r0", 50), ("r2", 2), ("r4", 1), ("r3", 33)])       # r2 and r4 end: two slots free
    run([("r0", 1), ("r3", 1), ("r5", 64)])
    while any(at[r] < len(toks[r]) for r in ("r0", "r3", "r5")):
        run([("r0", 1), ("r3", 7), ("r5", 2)])
        run([("r0", 37), ("r3", 1), ("r5", 1)])
    for rid in toks:
        _check(case, drv, rid)
    assert drv.runner.cache.stats()["state_slots_free"] == 4


def test_recorded_decode_steps_equal_eager_ones(case):
    """Three requests decode side by side for 50 steps, once step by step and once with recorded steps switched on (one
    request ends on the way, so the recorded size changes): the same logits (32-bit: the same bits)."""
    from infinilm_amd.engine.loading import load_model, make_runner
    from infinilm_amd.engine.step import StepEntry
    if case["page"] != 64:
        pytest.skip("one page size is enough here")
    toks = case["toks"]
    model = load_model(case["dir"], case["dtype"], DEV)
    ids = ["r0", "r3", "r5"]
    start = {"r0": 170, "r3": 30, "r5": 61}
    got = {}
    for graph in (False, True):
        runner = make_runner(model, num_pages=12, page_size=64, max_requests=4, enable_graph=graph)
        for r in ids:
            runner.cache.admit(r)
        runner.step([StepEntry(r, toks[r][:start[r]], []) for r in ids])
        rows = {r: [] for r in ids}
        for i in range(50):
            live = [r for r in ids if start[r] + i < len(toks[r])]
            out = runner.step([StepEntry(r, [toks[r][start[r] + i]], [0]) for r in live]).cpu()
            for j, r in enumerate(live):
                rows[r].append(out[j].clone())
            for r in live:
                if start[r] + i + 1 == len(toks[r]):
                    runner.cache.release(r)
        if graph:
            assert runner._graphs, "no step was recorded"
        got[graph] = {r: torch.stack(rows[r]) for r in ids}
    for r in ids:
        if case["dtype"] == "float32":
            assert torch.equal(got[True][r], got[False][r]), f"{r}: a recorded step differs from the eager one"
            want = P.forward(case["cfg"], case["W"], toks[r])
            _close(got[True][r], want[start[r]:start[r] + len(got[True][r])], TOL["float32"], f"{r} against the plain implementation")
        else:
            _close(got[True][r], got[False][r], TOL["bfloat16"], f"{r}: recorded against eager")


def test_logits_do_not_depend_on_the_cut_in_32_bit(case):
    if case["dtype"] != "float32":
        pytest.skip("the 32-bit path")
    page, toks = case["page"], case["toks"]
    a = Driver(case["dir"], "float32", num_pages=_pages(131, page) + 1, page_size=page, max_requests=2)
    a.step([("r5", toks["r5"])])
    b = Driver(case["dir"], "float32", num_pages=_pages(131, page) + _pages(70, page) + 2, page_size=page, max_requests=2)
    b.step([("r3", toks["r3"][:9]), ("r5", toks["r5"][:50])])
    b.step([("r5", toks["r5"][50:52]), ("r3", toks["r3"][9:])])
    b.step([("r5", toks["r5"][52:130])])
    b.step([("r5", toks["r5"][130:])])
    _close(b.request_logits("r5", 131), a.request_logits("r5", 131), 6e-6, "cut and batched against whole")


# ---- random configurations -----------------------------------------------------------------------------------------------
def _random_config(seed, widths=(24, 40, 64, 72, 96)):
    g = torch.Generator().manual_seed(3000 + seed)
    ri = lambda lo, hi: int(torch.randint(lo, hi + 1, (1,), generator=g))
    pick = lambda xs: xs[ri(0, len(xs) - 1)]

    def mlp():
        kind = ri(0, 3)
        if kind == 0:
            return None
        if kind == 1:
            return P.dense_mlp(pick([8, 30, 64, 100]))
        count, size = pick([1, 2, 3, 4]), ri(1, 4)
        total = count * size
        ident = ri(0, total - 1)
        keep = ri(1, count)
        return P.moe_mlp(total - ident, ident, ri(1, min(4, keep * size)), pick([8, 24, 33]), pick([0, 16, 21]),
                         (count, keep) if count > 1 or ri(0, 1) else None, pick([0.5, 1.0, 2.5]))

    layers = []
    for _ in range(ri(2, 5)):
        kind = pick(["attention", "attention_2", "mlstm"])
        if kind == "mlstm":
            layers.append(P.mlstm_layer(ri(1, 5), pick([4, 6, 10, 16, 32, 40]), pick([3, 7, 12, 16, 32]), pick([2.0, 8.0, 15.0, 40.0]), mlp()))
            continue
        G, dim = pick([1, 2, 3]), pick([4, 6, 10, 16, 32, 40])
        scaling = (pick([1.5, 4.0, 16.0]), pick([20, 64, 1000]), pick([8.0, 32.0]), pick([0.5, 1.0, 2.0])) if ri(0, 1) else None
        layers.append(P.attention_layer(kind, G * pick([1, 2, 3]), G, dim, dim if kind == "attention_2" else pick([4, 7, 12, 16, 32]),
                                        pick([10.0, 1000.0, 50000.0]), 2 * ri(0, dim // 2), mlp(), scaling, pick([None, 3.0, 50.0]), 0.7 / math.sqrt(dim)))
    cfg = {"architecture": "Lizezen", "vocab": pick([31, 64, 257]), "width": pick(list(widths)), "norm": {"eps": pick([1e-5, 1e-6, 1e-3])}, "layers": layers}
    if ri(0, 2):
        a = ri(0, len(layers) - 1)
        cfg["loop"] = {"start": a, "stop": ri(a + 1, len(layers)), "times": ri(1, 3)}
    return cfg


@pytest.mark.parametrize("seed,dtype", [(s, "float32") for s in range(20)] + [(s, "bfloat16") for s in range(20, 32)]
                         + [(s, "float32" if s % 2 else "bfloat16") for s in range(32, 44)])
def test_random_configurations(seed, dtype, tmp_path):
    """Layer order, every size, routers, loops; the last twelve with widths that are no multiples of 8 (or of 4).  Mixed steps with
    two slots and few pages."""
    cfg = _random_config(seed) if seed < 32 else _random_config(seed, widths=(20, 36, 50, 100, 132, 17))
    page = [4, 16, 64, 32][seed % 4]
    d = str(tmp_path / "m")
    W = make_dir(d, cfg, P.random_weights(cfg, seed), dtype)
    toks = {"a": tokens(cfg, 120, seed), "b": tokens(cfg, 40, seed + 1), "c": tokens(cfg, 3, seed + 2)}
    drv = RoutedDriver(d, dtype, num_pages=_pages(120, page) + _pages(40, page) + 2, page_size=page, max_requests=2)
    drv.step([("a", toks["a"][:70]), ("c", toks["c"][:2])])
    drv.step([("a", toks["a"][70:72]), ("c", toks["c"][2:])], end=["c"])
    drv.step([("a", toks["a"][72:73]), ("b", toks["b"][:33])])
    for i in range(73, 80):
        drv.step([("a", [toks["a"][i]]), ("b", [toks["b"][33 + i - 73]])], end=["b"] if i == 79 else [])
    drv.step([("a", toks["a"][80:])], end=["a"])
    for rid, t in toks.items():
        _compare(cfg, W, t, drv, rid, dtype, f"seed {seed} {rid} {json.dumps(cfg)}")


# ---- through the entry point ---------------------------------------------------------------------------------------------
@pytest.mark.parametrize("name,graph", [("A", False), ("B", True), ("C", True)])
def test_greedy_generation_through_the_entry_point(name, graph, tmp_path):
    """`LLM.generate` with its scheduler (three slots, portions of five tokens): every request token for token as the plain
    implementation generates it greedily."""
    from infinilm_amd import LLM, SamplingParams
    cfg = P.CONFIGS[name]()
    W = make_dir(str(tmp_path), cfg, P.random_weights(cfg, 77), "float32")
    prompts = [tokens(cfg, n, 5 + n) for n in (3, 40, 9, 50, 1)]
    llm = LLM(str(tmp_path), dtype="float32", num_blocks=24, block_size=16, max_batch_size=3, chunk_size=5,
              max_num_batched_tokens=11, enable_graph=graph)
    outs = llm.generate(prompt_token_ids=prompts, sampling_params=SamplingParams(top_k=1, max_tokens=10))
    for prompt, out in zip(prompts, outs):
        assert out.outputs[0].token_ids == P.greedy(cfg, W, prompt, 10), f"prompt of {len(prompt)} tokens"
    llm.close()


def test_recorded_steps_with_long_portions(tmp_path):
    """Portions of up to 160 tokens (chunks of the recurrence) in recorded steps that are replayed with other requests' portions of
    other lengths, decode steps recorded before the first request: greedy tokens as the plain implementation's."""
    from infinilm_amd import LLM, SamplingParams
    cfg = P.CONFIGS["C"]()
    W = make_dir(str(tmp_path), cfg, P.random_weights(cfg, 78), "float32")
    prompts = [tokens(cfg, n, 9 + n) for n in (200, 170, 129, 5, 161, 220)]
    llm = LLM(str(tmp_path), dtype="float32", num_blocks=40, block_size=32, max_batch_size=3, chunk_size=160,
              max_num_batched_tokens=192, enable_graph=True, record_graphs_at_start=True)
    outs = llm.generate(prompt_token_ids=prompts, sampling_params=SamplingParams(top_k=1, max_tokens=4))
    for prompt, out in zip(prompts, outs):
        assert out.outputs[0].token_ids == P.greedy(cfg, W, prompt, 4), f"prompt of {len(prompt)} tokens"
    llm.close()


def test_long_decoding(tmp_path):
    """500 decoded tokens after a prompt of 10 in recorded steps."""
    from infinilm_amd.engine.loading import load_model, make_runner
    from infinilm_amd.engine.step import StepEntry
    cfg = P.CONFIGS["A"]()
    d = str(tmp_path / "m")
    W = make_dir(d, cfg, P.random_weights(cfg, 3), "float32")
    toks = tokens(cfg, 510, 2)
    want = P.forward(cfg, W, toks)
    runner = make_runner(load_model(d, "float32", DEV), num_pages=32, page_size=16, max_requests=2, enable_graph=True)
    runner.cache.admit("a")
    runner.step([StepEntry("a", toks[:10], [])])
    rows = [runner.step([StepEntry("a", [toks[i]], [0])]).cpu()[0] for i in range(10, 510)]
    _close(torch.stack(rows), want[10:], TOL["float32"], "500 decoded tokens")
    runner.cache.check()
