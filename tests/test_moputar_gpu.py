"""The Moputar design in the engine against the plain implementation (`plain_moputar.py`): the new kernels alone, every
mechanism alone in a one-layer model (with a key made to stand out at chunk edges, page borders and a sequence's start), then
whole models through the engine's own step function (whole prompts, decoding token by token, portions down to two tokens, mixed
batches with pages and slots used again, recorded steps) and through the entry point with its scheduler (greedy generation).
Configurations A, B and C differ in every size and switch: 1, 3 and 6 streams, heads of 7 to 128 entries, convolutions of 1 to 8
taps and none, chunks of 20 to 96 positions and none, readers whose chunks differ from their writers', layers without a
feed-forward, without rotation."""
import copy
import json
import math
import os

import pytest
import torch

import plain_moputar as P
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


def _segments(lens):
    off, seg = [0], []
    for r, n in enumerate(lens):
        off.append(off[-1] + n)
        seg += [r] * n
    return i32(*off), i32(*seg)


# ---- the kernels alone ------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("n,H,T,parts,ydt,out", [(4, 352, 5, 1, "bfloat16", "bfloat16"), (1, 52, 3, 1, "float32", "float32"), (3, 61, 7, 3, "float32", "float32"),
                                                 (6, 4096, 33, 4, "float32", "bfloat16"), (2, 2304, 9, 16, "float32", "bfloat16"),
                                                 (16, 40, 4, 1, "bfloat16", "bfloat16"), (4, 4096, 1100, 1, "bfloat16", "bfloat16"), (11, 64, 2, 2, "float32", "float32")])
def test_hyper_update(K, n, H, T, parts, ydt, out):
    g = torch.Generator().manual_seed(n * H)
    rnd = lambda *s: torch.randn(s, generator=g)
    base, X = rnd(T, H), rnd(T, n, H)
    y = rnd(parts, T, H).to(getattr(torch, ydt))
    M, b, a, w = rnd(n, n), rnd(n), rnd(n), (0.3 * rnd(H)).to(getattr(torch, out))
    out = getattr(torch, out)
    d = lambda t: t.to(DEV)
    branch = d(y if parts > 1 else y[0])
    tol = 2e-6 if out == F32 else 6e-3
    for start in ("base", "streams"):
        old = base.double()[None].repeat(n, 1, 1) if start == "base" else X.double().transpose(0, 1)
        new = P.write_streams(old, M.double(), b.double(), 0.7 * y.double().sum(0))
        for weighted in (True, False):
            u = P.read_streams(new, a.double() if weighted else torch.ones(n, dtype=F64))
            want = P.rms(u, 1e-5) * (1 + w.double())
            for write in (True, False):
                dst = torch.full((T, n, H), 7.0, device=DEV) if start == "base" else d(X).clone()
                before = dst.clone()
                x = K.hyper_update(dst, n, base=d(base) if start == "base" else None, branch=branch, alpha=0.7, mix=d(M), out_weights=d(b),
                                   in_weights=d(a) if weighted else None, weight=d(w), weight_offset=1.0, eps=1e-5, out_dtype=out, write=write)
                _close(x, want, tol, f"{start} read")
                if write:
                    _close(dst.transpose(0, 1), new, 2e-6, f"{start} streams")
                else:
                    assert torch.equal(dst, before)
        # a read without a branch, and without a norm
        src = None if start == "base" else d(X).clone()
        u0 = P.read_streams(old, a.double())
        x = K.hyper_update(src, n, base=d(base) if start == "base" else None, in_weights=d(a), weight=d(w), weight_offset=1.0, eps=1e-5, out_dtype=out)
        _close(x, P.rms(u0, 1e-5) * (1 + w.double()), tol, f"{start} plain read")
        _close(K.hyper_update(src, n, base=d(base) if start == "base" else None, out_dtype=F32), old.sum(0), 2e-6, f"{start} sum")
    # a row does not depend on its batch
    if T > 4:
        one = K.hyper_update(d(X[2:3]).clone(), n, branch=branch[..., 2:3, :].contiguous(), mix=d(M), out_weights=d(b), in_weights=d(a), weight=d(w), weight_offset=1.0,
                             eps=1e-5, out_dtype=out)
        few = K.hyper_update(d(X[:4]).clone(), n, branch=branch[..., :4, :].contiguous(), mix=d(M), out_weights=d(b), in_weights=d(a), weight=d(w), weight_offset=1.0,
                             eps=1e-5, out_dtype=out)
        assert torch.equal(one[0], few[2])


@pytest.mark.parametrize("H", [64, 100, 4096, 51])
def test_norm_weights_around_zero(K, H):
    """The offset in the residual norm (both forms, few rows with many parts too) and in the norm of plain rows; a plain residual
    stream whose norm, branch norm or tail would otherwise be fused goes through the kernels that know the offset."""
    from infinilm_amd.parts import BuildContext, ResidualStream
    from infinilm_amd.parts.norm import RMSNorm
    g = torch.Generator().manual_seed(H)
    r, w = torch.randn((6, H), generator=g), 0.3 * torch.randn((H,), generator=g)
    for parts, dt in ((1, F32), (6, BF)):
        y = torch.randn((parts, 6, H), generator=g)
        want = P.rms(r.double() + 0.5 * y.double().sum(0), 1e-5) * (1 + w.double())
        x = K.add_rmsnorm(r.to(DEV).clone(), y.to(DEV) if parts > 1 else y[0].to(DEV), w.to(DEV), 0.5, 1e-5, dt, weight_offset=1.0)
        _close(x, want, 2e-6 if dt == F32 else 6e-3, "add_rmsnorm")
    _close(K.group_norm_gate(r.to(DEV), w.to(DEV), 1e-5, 1, out_dtype=F32, weight_offset=1.0), P.rms(r.double(), 1e-5) * (1 + w.double()), 2e-6, "plain rows")
    ctx = BuildContext(dtype=F32, device=torch.device(DEV))
    norm, post = RMSNorm(H, 1e-5, ctx, weight_offset=1.0), RMSNorm(H, 1e-6, ctx, weight_offset=1.0)
    norm.weight.copy_(w)
    post.weight.copy_(-w)
    s = ResidualStream(r.to(DEV).clone())
    y = torch.randn((6, H), generator=g)
    s.push_normed(y.to(DEV), post, 0.5)
    want = P.rms(r.double() + 0.5 * P.rms(y.double(), 1e-6) * (1 - w.double()), 1e-5) * (1 + w.double())
    assert norm.tail(s, 1.0, 6) is None
    _close(norm.forward(s), want, 4e-6, "a normed branch and the norm")
    s = ResidualStream(r.to(DEV).clone())
    s.push_normed(y.to(DEV), post, 0.5)
    _close(s.rows(F32), r.double() + 0.5 * P.rms(y.double(), 1e-6) * (1 - w.double()), 4e-6, "rows of a stream with a normed branch")


def test_one_weight_for_all_groups(K):
    g = torch.Generator().manual_seed(1)
    for n, groups in ((96, 6), (64, 4), (1024, 8), (60, 4), (256, 1), (600, 2)):
        x, w, gate = torch.randn((5, n), generator=g), torch.randn((n // groups,), generator=g), torch.randn((5, n), generator=g)
        want = (P.rms(x.double().view(5, groups, -1), 1e-5) * w.double()).reshape(5, n) * P.silu(gate.double())
        _close(K.group_norm_gate(x.to(DEV), w.to(DEV), 1e-5, groups, gate=gate.to(DEV), gate_act="silu"), want, 3e-6, f"{n} in {groups}")


@pytest.mark.parametrize("M,I,Kd", [(3, 48, 64), (8, 4096, 256), (24, 1000, 128), (40, 12288, 128), (300, 96, 64)])
def test_gelu_gate_in_every_form(K, M, I, Kd):
    g = torch.Generator().manual_seed(M)
    x, w = torch.randn((M, Kd), generator=g).to(BF), (torch.randn((2 * I, Kd), generator=g) / math.sqrt(Kd)).to(BF)
    gu = (x.double() @ w.double().T)
    for act, f in (("gelu_tanh", P.gelu_tanh), ("silu", P.silu)):
        want = f(gu[:, :I]) * gu[:, I:]
        got = K.gateup_swiglu_gemm(x.to(DEV), w.to(DEV), None, act=act)
        if got is not None:
            _close(got, want, 2e-2, f"fused {act}")
        for dt in (F32, BF):
            rows = gu.to(dt)
            r = rows.double()
            _close(K.swiglu(rows.to(DEV), act), f(r[:, :I]) * r[:, I:], 3e-6 if dt == F32 else 1e-2, f"{act} {dt}")
            odd = rows[:, 1:2 * I - 1].contiguous()      # no multiple of 8
            o = odd.double()
            _close(K.swiglu(odd.to(DEV), act), f(o[:, :I - 1]) * o[:, I - 1:], 3e-6 if dt == F32 else 1e-2, f"{act} {dt} odd")
    with pytest.raises(K.KernelError):
        K.swiglu(gu.float().to(DEV), "relu2")


def _conv_reference(x, w, hist, lens):
    """x [T, C], w [taps, C], hist: per segment the inputs before it [any, C] -> y, and every segment's last taps - 1 inputs."""
    if w is None:
        return x.double(), None
    taps, ys, last, at = w.shape[0], [], [], 0
    for r, n in enumerate(lens):
        full = torch.cat([hist[r].double(), x[at:at + n].double()])
        ys.append(P.short_conv(full, w.double().T)[hist[r].shape[0]:])
        last.append(torch.cat([torch.zeros((taps, x.shape[1]), dtype=F64), full])[full.shape[0] + taps - (taps - 1):])
        at += n
    return torch.cat(ys), last


CONV = [(6, 2, 10, 14, 2), (4, 2, 16, 24, 4), (3, 1, 7, 9, 3), (2, 2, 64, 64, 8), (4, 4, 32, 16, 1), (2, 1, 128, 128, 0), (8, 4, 24, 40, 5)]


@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("H,G,dk,dv,taps", CONV)
def test_conv_delta_inputs(K, H, G, dk, dv, taps, dtype):
    """Two launches over three requests (a fresh one, one that goes on, one token and many), the second step's states from rows the
    first wrote; then a launch of single tokens alone, which shifts the rows in the kernel itself."""
    g = torch.Generator().manual_seed(H * dk)
    hp = 8 * -(-H // 8)
    C, N = 2 * G * dk + H * dv, 2 * G * dk + 2 * H * dv + 2 * hp
    w = (0.5 * torch.randn((taps, C), generator=g)).to(dtype) if taps else None
    a_log, dt_bias = torch.randn((H,), generator=g), torch.randn((H,), generator=g)
    pool = torch.randn((6, max(taps - 1, 0), C), generator=g)
    pool[0] = 0
    pool = pool.to(DEV)
    hist = [torch.zeros((0, C)) for _ in range(3)]
    for step, lens in enumerate(((5, 1, 70), (1, 1, 1), (2, 300, 1), (1, 1, 1))):
        off, seg = _segments(lens)
        T = sum(lens)
        x = torch.randn((T, N), generator=g).to(dtype)
        sin, sout = (i32(0, 0, 0) if step == 0 else i32(2, 4, 1)), i32(2, 4, 1)
        rows, gates = K.conv_delta_inputs(x.to(DEV), w.to(DEV) if taps else None, pool, sin, sout, seg, off, 3, H, G, dk, dv, C + H * dv, C + H * dv + hp,
                                          a_log.to(DEV), dt_bias.to(DEV), 0.3, 1e-6, max_len=max(lens))
        y, last = _conv_reference(x[:, :C], w, hist, lens)
        y = P.silu(y)
        unit = lambda u: (u.view(T, G, dk) / torch.sqrt((u.view(T, G, dk) ** 2).sum(-1, keepdim=True) + 1e-6))
        dkp = -(-dk // 16) * 16
        got = rows.cpu().double()
        q, k, v = got[:, :G * dkp].view(T, G, dkp), got[:, G * dkp:2 * G * dkp].view(T, G, dkp), got[:, 2 * G * dkp:2 * G * dkp + H * dv]
        assert (q[..., dk:] == 0).all() and (k[..., dk:] == 0).all()
        _close(q[..., :dk], unit(y[:, :G * dk]) * 0.3, 3e-6, f"q step {step}")
        _close(k[..., :dk], unit(y[:, G * dk:2 * G * dk]), 3e-6, f"k step {step}")
        _close(v, y[:, 2 * G * dk:], 3e-6, f"v step {step}")
        xb, xa = x[:, C + H * dv:C + H * dv + H].double(), x[:, C + H * dv + hp:C + H * dv + hp + H].double()
        _close(gates[:, :H], torch.sigmoid(xb), 1e-6, "beta")
        _close(gates[:, H:], -torch.exp(a_log.double()) * torch.nn.functional.softplus(xa + dt_bias.double()), 1e-6, "log-decay")
        at = 0
        for r, n in enumerate(lens):
            hist[r] = torch.cat([hist[r], x[at:at + n, :C].float()])
            at += n
            if taps > 1:
                assert torch.equal(pool[[2, 4, 1][r]].cpu().double(), last[r]), f"state row of request {r} after step {step}"
    assert taps <= 1 or (pool[0] == 0).all()


@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("H,G,dim,vdim,rd,taps,own", [(4, 2, 12, 20, 6, 3, True), (6, 2, 64, 48, 24, 4, True), (4, 4, 16, 16, 16, 2, False), (3, 1, 7, 9, 0, 0, True),
                                                      (6, 3, 32, 48, 2, 1, True), (2, 1, 128, 128, 128, 8, True), (8, 1, 24, 16, 8, 5, False)])
def test_conv_norm_rope_kvwrite(K, H, G, dim, vdim, rd, taps, own, dtype):
    g = torch.Generator().manual_seed(H * dim + taps)
    C = H * dim + (G * (dim + vdim) if own else 0)
    d, page = -(-max(dim, vdim) // 16) * 16, 16
    w = (0.5 * torch.randn((taps, C), generator=g)).to(dtype) if taps else None
    wq, wk = torch.randn((H * dim,), generator=g).to(dtype), torch.randn((G * dim,), generator=g).to(dtype)
    freq = (1000.0 ** (-2.0 * torch.arange(rd // 2, dtype=F64) / rd)).float().to(DEV) if rd else None
    pool = torch.zeros((6, max(taps - 1, 0), C), device=DEV)
    kc, vc = torch.zeros((12, G, page, d), dtype=dtype, device=DEV), torch.zeros((12, G, d, page), dtype=dtype, device=DEV)
    hist, pos0 = [torch.zeros((0, C)) for _ in range(2)], [0, 0]
    x_all = []
    for step, lens in enumerate(((40, 1), (1, 3), (1, 1))):
        off, seg = _segments(lens)
        T = sum(lens)
        x = torch.randn((T, C + 8), generator=g).to(dtype)
        pos = torch.cat([torch.arange(pos0[r], pos0[r] + n) for r, n in enumerate(lens)]).to(torch.int32)
        slots = torch.tensor([(r * 5 + int(p) // page) * page + int(p) % page for r, n in enumerate(lens) for p in range(pos0[r], pos0[r] + n)], dtype=torch.int32)
        q = K.conv_norm_rope_kvwrite(x.to(DEV), w.to(DEV) if taps else None, pool, i32(0, 0) if step == 0 else i32(3, 1), i32(3, 1), seg, off, 2, pos.to(DEV), freq,
                                     wq.to(DEV), wk.to(DEV) if own else None, kc, vc, slots.to(DEV), H, G, dim, vdim, rd, 1e-5, own_kv=own, max_len=max(lens))
        y, last = _conv_reference(x[:, :C], w, hist, lens)
        rot = {"dims": rd, "base": 1000.0}
        tol = 5e-6 if dtype == F32 else 8e-3
        want_q = P.rotate_pairs((P.rms(y[:, :H * dim], 1e-5) * wq.double()).view(T, H, dim), pos, rot)
        _close(q.view(T, H, d)[..., :dim], want_q, tol, f"q step {step}")
        assert (q.view(T, H, d)[..., dim:] == 0).all()
        if own:
            want_k = P.rotate_pairs((P.rms(y[:, H * dim:(H + G) * dim], 1e-5) * wk.double()).view(T, G, dim), pos, rot)
            pg, of = slots.long() // page, slots.long() % page
            _close(kc.cpu()[pg, :, of][..., :dim], want_k, tol, f"k step {step}")
            _close(vc.cpu()[pg, :, :, of][..., :vdim], y[:, (H + G) * dim:].view(T, G, vdim), tol, f"v step {step}")
        else:
            assert (kc == 0).all() and (vc == 0).all()
        at = 0
        for r, n in enumerate(lens):
            hist[r] = torch.cat([hist[r], x[at:at + n, :C].float()])
            at, pos0[r] = at + n, pos0[r] + n
            if taps > 1:
                assert torch.equal(pool[[3, 1][r]].cpu().double(), last[r])


DELTA = [(6, 2, 10, 14), (2, 2, 64, 64), (4, 1, 128, 128), (3, 3, 7, 9), (2, 1, 48, 80), (1, 1, 1, 1), (2, 1, 100, 20), (4, 2, 16, 200), (1, 1, 256, 40), (2, 1, 128, 300), (1, 1, 500, 33)]


@pytest.mark.parametrize("H,G,dk,dv", DELTA)
def test_delta_rule_kernels(K, H, G, dk, dv):
    """Four launches over four requests whose states pass through pool rows that were used before: long and short segments
    together (chunks and single steps side by side), lengths at and around chunk edges, single tokens, decays from none to total."""
    g = torch.Generator().manual_seed(H * dk + dv)
    dkp = -(-dk // 16) * 16
    pool = torch.randn((8, H, dv, dk), generator=g)
    pool[0] = 0
    pool = pool.to(DEV)
    w, S = torch.randn((dv,), generator=g), [None] * 4
    for step, lens in enumerate(((64, 1, 200, 31), (1, 1, 1, 1), (65, 128, 2, 33), (3, 5, 1, 2))):
        off, seg = _segments(lens)
        T = sum(lens)
        q, k = (torch.nn.functional.normalize(torch.randn((T, G, dk), generator=g), dim=-1) for _ in range(2))
        if step == 0 and T > 100:
            k[70:100] = k[70]                         # one key again and again: the corrections' system at its stiffest
        v, gate = torch.randn((T, H, dv), generator=g), torch.randn((T, H * dv), generator=g)
        beta = torch.rand((T, H), generator=g)
        logg = -torch.exp(2.0 * torch.randn((T, H), generator=g) - 3.0)
        logg[::17] = -20.0                            # forgets everything
        logg[5::11] = 0.0                             # forgets nothing
        rows = torch.zeros((T, -(-(2 * G * dkp + H * dv) // 4) * 4))
        rows[:, :G * dkp].view(T, G, dkp)[..., :dk] = q * 0.4
        rows[:, G * dkp:2 * G * dkp].view(T, G, dkp)[..., :dk] = k
        rows[:, 2 * G * dkp:2 * G * dkp + H * dv] = v.view(T, -1)
        gates = torch.cat([beta, logg], 1)
        sin, sout = (i32(0, 0, 0, 0) if step == 0 else i32(5, 2, 7, 1)), i32(5, 2, 7, 1)
        y = K.delta_rule(rows.to(DEV), gates.to(DEV), H, G, dk, dv, pool, sin, sout, off, 4, w.to(DEV), gate.to(DEV), 1e-5, F32, max_len=max(lens))
        at = 0
        for r, n in enumerate(lens):
            c = slice(at, at + n)
            o, S[r] = P.delta_rule(0.4 * q[c].double(), k[c].double(), v[c].double(), torch.exp(logg[c].double()), beta[c].double(), S[r])
            want = P.rms(o, 1e-5) * w.double() * P.silu(gate[c].double()).view(n, H, dv)
            _close(pool[[5, 2, 7, 1][r]].transpose(1, 2), S[r], 1e-5, f"state of request {r} after step {step}")
            # (the norm magnifies what is left of an output near zero: compared where the design compares it, after it)
            _close(y[c].view(n, H, dv), want, 2e-5 if dv > 2 else 2e-3, f"outputs of request {r} step {step}")
            at += n
    assert (pool[0] == 0).all()


def test_delta_rule_chunks_and_steps_agree(K):
    g = torch.Generator().manual_seed(3)
    H, G, dk, dv, T = 4, 2, 64, 32, 300
    rows, gates = torch.randn((T, 2 * G * dk + H * dv), generator=g), torch.cat([torch.rand((T, H), generator=g), -0.1 * torch.rand((T, H), generator=g)], 1)
    kk = rows[:, G * dk:2 * G * dk].view(T, G, dk)
    kk /= kk.norm(dim=-1, keepdim=True)
    w, gate = torch.ones((dv,), device=DEV), torch.randn((T, H * dv), generator=g).to(DEV)
    res = []
    for max_len in (T, None):
        pool = torch.zeros((3, H, dv, dk), device=DEV)
        y = K.delta_rule(rows.to(DEV), gates.to(DEV), H, G, dk, dv, pool, i32(0), i32(2), i32(0, T), 1, w, gate, 1e-5, F32, max_len=max_len)
        res.append((y, pool[2]))
    _close(res[0][0], res[1][0], 2e-5, "outputs")
    _close(res[0][1], res[1][1], 1e-5, "state")


@pytest.mark.parametrize("dtype,nh,nkv,d,page", [("bfloat16", 8, 4, 64, 64), ("bfloat16", 4, 2, 128, 64), ("bfloat16", 6, 3, 48, 16), ("bfloat16", 20, 1, 32, 32), ("float32", 6, 2, 64, 64),
                                                 ("float32", 4, 2, 128, 16), ("float32", 3, 3, 12, 4), ("bfloat16", 2, 2, 24, 8), ("bfloat16", 4, 1, 128, 16)])
@pytest.mark.parametrize("chunk", [1, 7, 40, 64, 100, 256])
def test_attention_by_chunks(K, dtype, nh, nkv, d, page, chunk):
    """One request of 300 tokens on shuffled pages: tiles of eight that straddle chunk edges, and every token alone.  Random keys,
    and one key of a score that outweighs all others at every place next to a chunk's edge in turn: it must show in full to its own
    chunk and not at all to the next.  Weights close to one another at a hundred keys show whether they stay float."""
    n = 300
    dt = getattr(torch, dtype)
    g = torch.Generator().manual_seed(nh * d + chunk)
    q, k, v = (torch.randn((n, h, d), generator=g).to(dt) for h in (nh, nkv, nkv))
    pages = -(-n // page)
    order = torch.randperm(pages + 2, generator=g)[:pages]
    pos = torch.arange(n, dtype=torch.int32)
    tiles = torch.tensor([[t, min(8, n - t)] for t in range(0, n, 8)], dtype=torch.int32, device=DEV)
    mask = P.visible(n, chunk)
    for mark in (None, chunk - 1, chunk, 2 * chunk - 1, (n // chunk) * chunk - 1, 255, 256):
        if mark is not None and not 0 <= mark < n:
            continue
        kk = k.clone()
        if mark is not None:
            kk[mark] = 6.0 * q.view(n, nkv, nh // nkv, d).float().mean((0, 2)).to(dt) + 0.0   # a key along ...
            qq = q.clone()
            qq[:, :, :] = (q.float() * 0.05 + kk[mark].float().repeat_interleave(nh // nkv, 0)[None] * 3.0).to(dt)    # ... every query
        else:
            qq = q
        kc, vc = torch.zeros((pages + 2, nkv, page, d), dtype=dt), torch.zeros((pages + 2, nkv, d, page), dtype=dt)
        for j in range(n):
            kc[order[j // page], :, j % page] = kk[j]
            vc[order[j // page], :, :, j % page] = v[j]
        want = P.softmax_attention(qq.double(), kk.double(), v.double(), 0.3, mask).reshape(n, -1)
        dev = (qq.reshape(n, -1).contiguous().to(DEV), kc.to(DEV), vc.to(DEV), order.to(torch.int32)[None].contiguous().to(DEV))
        sg = torch.zeros((n,), dtype=torch.int32, device=DEV)
        tol = 4e-6 if dtype == "float32" else 6e-3
        for name, tl in (("tiles", tiles), ("single tokens", None)):
            o = K.paged_attention(*dev, sg, pos.to(DEV), nh, nkv, d, 0.3, 0, n, tl, None, float_weights=True, chunk=chunk)
            _close(o, want, tol, f"{name}, marked key {mark}")


def test_a_window_and_a_chunk_exclude_each_other(K):
    z = torch.zeros((1, 16), device=DEV)
    c = torch.zeros((1, 1, 16, 16), device=DEV)
    with pytest.raises(K.KernelError):
        K.paged_attention(z, c, c, i32(0).view(1, 1), i32(0), i32(0), 1, 1, 16, 1.0, window=4, chunk=4)


def test_softmax_weights_stay_float(K):
    """1,024 keys whose weights lie close to one another, and values that cancel but for the differences: rounding the weights costs
    far more than float weights lose (portions and decoded tokens, heads of 64 and 128)."""
    for d in (64, 128):
        g = torch.Generator().manual_seed(d)
        n, page, nh = 1024, 64, 4
        q = torch.randn((8, nh, d), generator=g).to(BF)
        k = (0.02 * torch.randn((n, 1, d), generator=g)).to(BF)
        v = torch.randn((n, 1, d), generator=g)
        v = (v - v.mean(0)).to(BF)
        kc, vc = k.view(n // page, page, 1, d).transpose(1, 2).contiguous(), v.view(n // page, page, 1, d).permute(0, 2, 3, 1).contiguous()
        mask = torch.arange(n)[None, :] <= torch.arange(n - 8, n)[:, None]
        want = torch.zeros((8, nh, d), dtype=F64)
        for h in range(nh):
            s = (q[:, h].double() @ k[:, 0].double().T * 0.3).masked_fill(~mask, -math.inf)
            want[:, h] = torch.softmax(s, -1) @ v[:, 0].double()
        args = (q.reshape(8, -1).to(DEV), kc.to(DEV), vc.to(DEV), torch.arange(n // page, dtype=torch.int32, device=DEV)[None], torch.zeros((8,), dtype=torch.int32, device=DEV),
                torch.arange(n - 8, n, dtype=torch.int32, device=DEV), nh, 1, d, 0.3, 0, n)
        for tl in (i32(0, 8).view(1, 2), None):
            err = {fw: float((K.paged_attention(*args, tl, None, float_weights=fw).double().cpu().view(8, nh, d) - want).abs().max()) for fw in (True, False)}
            assert err[True] < 0.2 * err[False], err


# ---- one mechanism in a one-layer model ---------------------------------------------------------------------------------
def _one_layer(kind, mixer, mlp=None, streams=2):
    return {"architecture": "Moputar", "vocab": 50, "width": 48, "streams": streams, "embedding": {"scale": 1.0}, "norm": {"eps": 1e-5},
            "layers": [{"type": kind, "mixer": mixer, "mlp": mlp}]}


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("dim,vdim,page,chunk", [(16, 16, 16, 48), (64, 48, 64, 128), (12, 20, 4, 33), (64, 64, 64, 100)])
def test_a_key_at_a_chunks_edge(dim, vdim, page, chunk, dtype, tmp_path):
    """A token whose key outweighs all others for every query (its own embedding row makes it so), once next to every chunk edge and
    page border near 200, one position inside and outside: in a prompt, in portions and for decoded tokens."""
    mixer = {"heads": 4, "kv_heads": 2, "dim": dim, "vdim": vdim, "scale": 3.0 / math.sqrt(dim), "mask": {"size": chunk}}
    cfg = _one_layer("attention", mixer)
    W = P.random_weights(cfg, 5)
    g = torch.Generator().manual_seed(1)
    loud, all_dir, dirs = (torch.randn((n,), generator=g) for n in (48, 48, dim))
    W["embed"] = 0.3 * W["embed"] + all_dir          # every token's query holds `dirs`
    W["embed"][7] = 4.0 * loud                        # token 7's key does, and strongly
    W["l0.mix.q"] += (dirs.repeat(4)[:, None] * all_dir[None] / all_dir.norm() ** 2) * 3
    W["l0.mix.k"] += (dirs.repeat(2)[:, None] * loud[None] / loud.norm() ** 2) * 3
    W["l0.mix.q.norm"].fill_(1.0)
    W["l0.mix.k.norm"].fill_(1.0)
    base = [t if t != 7 else 8 for t in tokens(cfg, 240, 3)]
    edge = (200 // chunk) * chunk
    d = str(tmp_path / "m")
    Wr = make_dir(d, cfg, W, dtype)
    drv = Driver(d, dtype, num_pages=-(-240 // page) + 2, page_size=page, max_requests=2)
    quiet = P.forward(cfg, Wr, base)
    shown = 0
    for i, at in enumerate((edge - 1, edge, edge + 1, 192, 191, 0)):
        toks = list(base)
        toks[at] = 7
        want = P.forward(cfg, Wr, toks)
        seen = [j for j in range(at + 1, 240) if j // chunk == at // chunk]
        if seen:
            assert rel_err(want[seen], quiet[seen]) > 0.05, "the marked key does not show"
            shown += 1
        out = [j for j in range(at + 1, 240) if j // chunk != at // chunk]
        if out:
            assert rel_err(want[out], quiet[out]) < 1e-9
        rid = f"r{i}"
        cuts = [(240,), (150, 2, 50) + (1,) * 38, (197,) + (1,) * 43][i % 3]
        a = 0
        for n in cuts:
            drv.step([(rid, toks[a:a + n])], end=[rid] if a + n == 240 else [])
            a += n
        _close(drv.request_logits(rid, 240), want, TOL[dtype], f"marked key at {at}")
    assert shown >= 3


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_first_tokens_of_a_sequence(dtype, tmp_path):
    """The first tokens (zeros before the convolutions' start, a chunk of one key, an empty state), alone, in twos and whole, in
    slots and pages another request has used."""
    cfg = P.config_a()
    d = str(tmp_path / "m")
    W = make_dir(d, cfg, P.random_weights(cfg, 2), dtype)
    drv = Driver(d, dtype, num_pages=4, page_size=16, max_requests=1)
    drv.step([("x", tokens(cfg, 40, 9))], end=["x"])
    for i, cut in enumerate(((1,) * 6, (2, 2, 2), (6,), (1, 5), (3, 1, 2))):
        toks, a = tokens(cfg, 6, 20 + i), 0
        for n in cut:
            drv.step([(f"r{i}", toks[a:a + n])], end=[f"r{i}"] if a + n == 6 else [])
            a += n
        _compare(cfg, W, toks, drv.request_logits(f"r{i}", 6), dtype, f"cut {cut}")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("dim,vdim", [(10, 14), (64, 64), (128, 128), (160, 40)])
def test_delta_state_remembers_through_portions(dim, vdim, dtype, tmp_path):
    """Slow decays: a token as far back as keys of this size can remember (300 positions, or twice their size) still shows, through portions on either side of the chunks' length and decoded tokens."""
    cfg = _one_layer("delta", {"heads": 2, "kv_heads": 1, "dim": dim, "vdim": vdim, "conv": 3})
    W = P.random_weights(cfg, 9)
    W["l0.mix.A_log"] = torch.full_like(W["l0.mix.A_log"], -6.0)
    toks = tokens(cfg, 320, 4)
    d = str(tmp_path / "m")
    Wr = make_dir(d, cfg, W, dtype)
    want = P.forward(cfg, Wr, toks)
    other = list(toks)
    far = max(20, 320 - 2 * dim)
    other[far] = (toks[far] + 1) % cfg["vocab"]
    assert rel_err(P.forward(cfg, Wr, other)[-1], want[-1]) > 1e-4
    drv = Driver(d, dtype, num_pages=1, page_size=16, max_requests=2)
    at = 0
    for n in [2, 131, 3, 64, 31, 33, 30]:
        drv.step([("a", toks[at:at + n])])
        at += n
    for i in range(at, 320):
        drv.step([("a", [toks[i]])])
    _close(drv.request_logits("a", 320), want, TOL[dtype], "delta rule through portions")


def test_streams_mix_and_dump(tmp_path):
    """A mix matrix far from the identity and from symmetric (indexed from, to), and the dump of the streams' sum after every layer."""
    from infinilm_amd.engine.loading import load_model, make_runner
    from infinilm_amd.engine.step import StepEntry
    cfg = P.config_a()
    W = P.random_weights(cfg, 6)
    for i in range(4):
        W[f"l{i}.hc1.mix"] = torch.tensor([[0.2, 1.1, 0.0], [0.0, -0.3, 0.9], [0.8, 0.1, 0.4]])
    W = make_dir(str(tmp_path), cfg, W, "float32")
    model = load_model(str(tmp_path), "float32", DEV)
    runner = make_runner(model, num_pages=8, page_size=16, max_requests=2)
    toks = tokens(cfg, 30, 1)
    logits, layers = P.forward(cfg, W, toks, return_layers=True)
    runner.cache.admit("a")
    taps = {}
    got = runner.step([StepEntry("a", toks, [3, 29])], taps=taps)
    _close(got, logits[[3, 29]], TOL["float32"], "logits")
    for i in range(4):
        residual, pending, _ = taps[f"run{i}"]
        assert pending is None
        _close(residual, layers[i], TOL["float32"], f"streams' sum after layer {i}")


# ---- whole models through the step function -----------------------------------------------------------------------------
def _bound(cfg, W, toks, want, dtype):
    """float32: the tests' own; bfloat16: the other tests' 4e-2, or twice the error of the plain implementation with its projections'
    operands and results rounded where that is larger."""
    return TOL[dtype] if dtype == "float32" else max(TOL[dtype], 2.0 * rel_err(P.forward(cfg, W, toks, round_to=BF), want))


def _compare(cfg, W, toks, got, dtype, what):
    want = P.forward(cfg, W, toks)
    tol = _bound(cfg, W, toks, want, dtype)
    err = rel_err(got, want)
    print(f"[err] {what} {dtype} n={len(toks)}: {err:.3e} (bound {tol:.3e})")
    assert err < tol, f"{what} {dtype}: error {err:.3e} (bound {tol:.3e})"


CASES = [(c, d, p) for d in ("float32", "bfloat16") for c, p in (("A", 16), ("B", 64), ("C", 64), ("C", 32), ("A", 4))]


@pytest.fixture(scope="module", params=CASES, ids=[f"{c}-{d}-p{p}" for c, d, p in CASES])
def case(request, tmp_path_factory):
    name, dtype, page = request.param
    cfg = P.CONFIGS[name]()
    d = tmp_path_factory.mktemp(f"moputar_{name}_{dtype}")
    W = make_dir(str(d), cfg, P.random_weights(cfg, 40 + ord(name)), dtype)
    toks = {r: tokens(cfg, n, 11 * i + 3) for i, (r, n) in
            enumerate([("r0", 300), ("r1", 1), ("r2", 45), ("r3", 70), ("r4", 2), ("r5", 131)])}
    return {"cfg": cfg, "dir": str(d), "dtype": dtype, "toks": toks, "name": name, "page": page, "W": W}


def _check(case, drv, rid):
    n = len(case["toks"][rid])
    _compare(case["cfg"], case["W"], case["toks"][rid], drv.request_logits(rid, n), case["dtype"], f"{case['name']} {rid}")


def _pages(n, page):
    return -(-n // page)


def test_whole_requests(case):
    page = case["page"]
    drv = Driver(case["dir"], case["dtype"], num_pages=_pages(300, page) + 1, page_size=page, max_requests=2)
    for rid, t in case["toks"].items():
        drv.step([(rid, t)], end=[rid])
        _check(case, drv, rid)


def test_last_tokens_one_by_one(case):
    """The last 140 tokens decoded one by one (longer than every chunk, so chunk edges pass over decoded tokens)."""
    page = case["page"]
    drv = Driver(case["dir"], case["dtype"], num_pages=_pages(300, page) + 1, page_size=page, max_requests=2)
    for rid, t in case["toks"].items():
        head = max(len(t) - 140, 0)
        if head:
            drv.step([(rid, t[:head])])
        for i in range(head, len(t)):
            drv.step([(rid, [t[i]])], end=[rid] if i == len(t) - 1 else [])
        _check(case, drv, rid)


def test_portions_of_changing_size(case):
    page = case["page"]
    drv = Driver(case["dir"], case["dtype"], num_pages=_pages(300, page) + 1, page_size=page, max_requests=2)
    sizes = [2, 5, page, 3, 2 * page + 1, 2, 17, page - 1, 1, 64]
    for rid, t in case["toks"].items():
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
    drv = Driver(case["dir"], case["dtype"], num_pages=_pages(300, page) + _pages(131, page) + 3, page_size=page, max_requests=4)
    at = {r: 0 for r in toks}

    def take(rid, n):
        a = at[rid]
        at[rid] = min(a + n, len(toks[rid]))
        return (rid, toks[rid][a:at[rid]])

    def run(plan):
        entries = [take(r, n) for r, n in plan if at[r] < len(toks[r])]
        if entries:
            drv.step(entries, end=[r for r, _ in entries if at[r] == len(toks[r])])

    run([("r1", 1), ("r0", 100), ("r2", 3)])
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
    """Three requests decode side by side for 70 steps, once step by step and once with recorded steps switched on (one
    request ends on the way, so the recorded size changes): the same logits (32-bit: the same bits)."""
    from infinilm_amd.engine.loading import load_model, make_runner
    from infinilm_amd.engine.step import StepEntry
    if case["page"] != 64:
        pytest.skip("one page size is enough here")
    toks = case["toks"]
    model = load_model(case["dir"], case["dtype"], DEV)
    ids = ["r0", "r3", "r5"]
    start = {"r0": 200, "r3": 20, "r5": 61}
    got = {}
    for graph in (False, True):
        runner = make_runner(model, num_pages=12, page_size=64, max_requests=4, enable_graph=graph)
        for r in ids:
            runner.cache.admit(r)
        runner.step([StepEntry(r, toks[r][:start[r]], []) for r in ids])
        rows = {r: [] for r in ids}
        for i in range(70):
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
    _close(b.request_logits("r5", 131), a.request_logits("r5", 131), 4e-6, "cut and batched against whole")


# ---- random configurations -----------------------------------------------------------------------------------------------
def _random_config(seed, widths=(24, 40, 64, 72, 96)):
    g = torch.Generator().manual_seed(2000 + seed)
    ri = lambda lo, hi: int(torch.randint(lo, hi + 1, (1,), generator=g))
    pick = lambda xs: xs[ri(0, len(xs) - 1)]
    layers, writers = [], []
    for i in range(ri(2, 5)):
        kind = pick(["attention", "attention", "delta"])
        G = pick([1, 2, 3])
        dim = pick([4, 6, 10, 16, 32, 40])
        mixer = {"heads": G * pick([1, 2, 3]), "kv_heads": G, "dim": dim, "vdim": pick([4, 7, 12, 16, 32])}
        if kind == "delta":
            mixer["conv"] = ri(1, 8)
        else:
            mixer["scale"] = 0.5 / math.sqrt(dim)
            if ri(0, 3):
                mixer["rot"] = {"base": pick([10.0, 1000.0, 50000.0]), "dims": 2 * ri(1, dim // 2)}
            if ri(0, 3):
                mixer["conv"] = ri(1, 4)
            if writers and ri(0, 1):
                src = pick(writers)
                mixer = {k: v for k, v in layers[src]["mixer"].items() if k != "mask"}
                mixer["kv_from"] = src
            else:
                writers.append(i)
            if ri(0, 3):
                mixer["mask"] = {"size": pick([1, 2, 7, 30, 64, 100])}
        layers.append({"type": kind, "mixer": mixer, "mlp": {"kind": "dense", "ff": pick([8, 30, 64])} if ri(0, 2) else None})
    return {"architecture": "Moputar", "vocab": pick([31, 64, 257]), "width": pick(list(widths)), "streams": pick([1, 2, 3, 4, 5, 8]),
            "embedding": {"scale": pick([0.5, 1.0, 7.0])}, "norm": {"eps": pick([1e-5, 1e-6])}, "layers": layers}


@pytest.mark.parametrize("seed,dtype", [(s, "float32") for s in range(24)] + [(s, "bfloat16") for s in range(24, 36)]
                         + [(s, "float32" if s % 2 else "bfloat16") for s in range(36, 48)])
def test_random_configurations(seed, dtype, tmp_path):
    """Layer order, every size, readers with other chunks than their writers', 1 to 8 streams; the last twelve with widths that are
    no multiples of 8 (or of 4).  Mixed steps with two slots and few pages."""
    cfg = _random_config(seed) if seed < 36 else _random_config(seed, widths=(20, 36, 50, 100, 132, 17))
    page = [4, 16, 64, 32][seed % 4]
    d = str(tmp_path / "m")
    W = make_dir(d, cfg, P.random_weights(cfg, seed), dtype)
    toks = {"a": tokens(cfg, 150, seed), "b": tokens(cfg, 40, seed + 1), "c": tokens(cfg, 3, seed + 2)}
    drv = Driver(d, dtype, num_pages=_pages(150, page) + _pages(40, page) + 2, page_size=page, max_requests=2)
    drv.step([("a", toks["a"][:70]), ("c", toks["c"][:2])])
    drv.step([("a", toks["a"][70:72]), ("c", toks["c"][2:])], end=["c"])
    drv.step([("a", toks["a"][72:73]), ("b", toks["b"][:33])])
    for i in range(73, 80):
        drv.step([("a", [toks["a"][i]]), ("b", [toks["b"][33 + i - 73]])], end=["b"] if i == 79 else [])
    drv.step([("a", toks["a"][80:])], end=["a"])
    for rid, t in toks.items():
        _compare(cfg, W, t, drv.request_logits(rid, len(t)), dtype, f"seed {seed} {rid}")


# ---- through the entry point ---------------------------------------------------------------------------------------------
def _greedy(cfg, W, prompt, n):
    seq = list(prompt)
    for _ in range(n):
        seq.append(int(P.forward(cfg, W, seq)[-1].argmax()))
    return seq[len(prompt):]


@pytest.mark.parametrize("name,graph", [("A", False), ("B", True), ("C", True)])
def test_greedy_generation_through_the_entry_point(name, graph, tmp_path):
    """`LLM.generate` with its scheduler (three slots, portions of five tokens): every request token for token as the plain
    implementation generates it greedily."""
    from infinilm_amd import LLM, SamplingParams
    cfg = P.CONFIGS[name]()
    W = make_dir(str(tmp_path), cfg, P.random_weights(cfg, 77), "float32")
    prompts = [tokens(cfg, n, 5 + n) for n in (3, 40, 9, 64, 1)]
    llm = LLM(str(tmp_path), dtype="float32", num_blocks=24, block_size=16, max_batch_size=3, chunk_size=5,
              max_num_batched_tokens=11, enable_graph=graph)
    outs = llm.generate(prompt_token_ids=prompts, sampling_params=SamplingParams(top_k=1, max_tokens=12))
    for prompt, out in zip(prompts, outs):
        assert out.outputs[0].token_ids == _greedy(cfg, W, prompt, 12), f"prompt of {len(prompt)} tokens"
    llm.close()


def test_recorded_steps_with_long_portions(tmp_path):
    """Portions of up to 160 tokens (chunks of the recurrence) in recorded steps that are replayed with other requests' portions of
    other lengths, decode steps recorded before the first request: greedy tokens as the plain implementation's."""
    from infinilm_amd import LLM, SamplingParams
    cfg = P.CONFIGS["C"]()
    W = make_dir(str(tmp_path), cfg, P.random_weights(cfg, 78), "float32")
    prompts = [tokens(cfg, n, 9 + n) for n in (300, 170, 129, 5, 161, 320)]
    llm = LLM(str(tmp_path), dtype="float32", num_blocks=40, block_size=32, max_batch_size=3, chunk_size=160,
              max_num_batched_tokens=192, enable_graph=True, record_graphs_at_start=True)
    outs = llm.generate(prompt_token_ids=prompts, sampling_params=SamplingParams(top_k=1, max_tokens=6))
    for prompt, out in zip(prompts, outs):
        assert out.outputs[0].token_ids == _greedy(cfg, W, prompt, 6), f"prompt of {len(prompt)} tokens"
    llm.close()


def test_long_decoding(tmp_path):
    """600 decoded tokens after a prompt of 10, recorded steps, pages of 16 given back as the chunks pass: five pages are enough."""
    from infinilm_amd.engine.loading import load_model, make_runner
    from infinilm_amd.engine.step import StepEntry
    cfg = P.CONFIGS["A"]()
    d = str(tmp_path / "m")
    W = make_dir(d, cfg, P.random_weights(cfg, 3), "float32")
    toks = tokens(cfg, 610, 2)
    want = P.forward(cfg, W, toks)
    model = load_model(d, "float32", DEV)
    runner = make_runner(model, num_pages=5, page_size=16, max_requests=2, enable_graph=True)
    runner.cache.admit("a")
    runner.step([StepEntry("a", toks[:10], [])])
    rows = [runner.step([StepEntry("a", [toks[i]], [0])]).cpu()[0] for i in range(10, 610)]
    _close(torch.stack(rows), want[10:], TOL["float32"], "600 decoded tokens")
    runner.cache.check()
