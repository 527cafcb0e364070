"""Lizezen without a GPU: config.json's keys and their errors, the tensor names against the plain list, the cache entries of looped
runs, what config.json leaves out, the frequencies, the random weights' neutral values, and the plain implementation's own
consistency."""
import copy
import math

import pytest
import torch

import plain_lizezen as P
from infinilm_amd.cache import FixedState, PagedKV
from infinilm_amd.config.errors import ConfigError
from infinilm_amd.config.registry import load_model_config
from infinilm_amd.engine.model import CausalLM


def _build(cfg):
    arch, c = load_model_config(cfg)
    spec = arch.build_spec(c)
    return spec, CausalLM(spec, torch.bfloat16, "meta")


@pytest.mark.parametrize("name", ["A", "B", "C"])
def test_tensor_names_and_shapes(name):
    cfg = P.CONFIGS[name]()
    spec, model = _build(cfg)
    assert {k: tuple(p.shape) for k, p in model.named_parameters().items()} == P.tensor_shapes(cfg)
    assert spec.architecture == "Lizezen"


def test_order_of_runs_and_their_cache_entries():
    spec, model = _build(P.config_a())
    assert [(r.layer, r.cache, r.start is not None) for r in spec.order] == [(0, 0, True), (1, 1, False), (0, 2, True), (1, 3, False), (2, 4, False)]
    assert all(r.start.project_embedding for r in spec.order if r.start is not None)
    kv, mem = PagedKV(2, 32), (FixedState((3, 15, 10), torch.float32), FixedState((3,), torch.float32))
    assert model.cache_needs == [kv, mem, kv, mem, PagedKV(3, 32)]
    spec, model = _build(P.config_b())
    assert spec.run_projection is None and all(r.start is None for r in spec.order)
    spec, _ = _build(P.config_c())
    assert [(r.layer, r.start is not None) for r in spec.order] == [(0, False), (1, True), (1, True), (1, True), (2, False), (3, False)]


def test_what_config_leaves_out_does_not_exist():
    _, model = _build(P.config_b())
    assert model.run_projection is None
    ffn = model.blocks[0].ffn
    assert ffn.identity == 0 and (ffn.groups, ffn.keep) == (1, 1) and ffn.shared is None
    assert model.blocks[1].mixer.softcap == 0.0 and model.blocks[2].mixer.softcap == 8.0
    assert model.blocks[2].mixer.position.rotary_dim == 0
    assert model.blocks[2].ffn is None
    cfg = P.config_b()
    del cfg["layers"][2]["mixer"]["rot"]
    cfg["loop"] = None
    _build(cfg)


@pytest.mark.parametrize("change,word", [
    (lambda c: c.pop("width"), "width"),
    (lambda c: c["norm"].pop("eps"), "eps"),
    (lambda c: c.__setitem__("layers", []), "layers"),
    (lambda c: c["layers"][0].__setitem__("type", "gla"), "gla"),
    (lambda c: c["layers"][0]["mixer"].__setitem__("kv_heads", 3), "kv_heads"),
    (lambda c: c["layers"][0]["mixer"].pop("scale"), "scale"),
    (lambda c: c["layers"][0]["mixer"]["rot"].__setitem__("dims", 14), "dims"),
    (lambda c: c["layers"][0]["mixer"]["rot"].__setitem__("dims", 7), "dims"),
    (lambda c: c["layers"][0]["mixer"]["rot"].pop("base"), "base"),
    (lambda c: c["layers"][1]["mixer"].pop("gate_cap"), "gate_cap"),
    (lambda c: c["layers"][1]["mixer"].__setitem__("gate_cap", 0.0), "gate_cap"),
    (lambda c: c["layers"][1]["mixer"].pop("vdim"), "vdim"),
    (lambda c: c["layers"][1]["mlp"].__setitem__("kind", "gated"), "gated"),
    (lambda c: c["layers"][1]["mlp"].pop("ff"), "ff"),
    (lambda c: c["layers"][2]["mixer"].__setitem__("vdim", 16), "16"),
    (lambda c: c["layers"][2]["mixer"]["rot"]["scaling"].pop("slow"), "slow"),
    (lambda c: c["layers"][2]["mixer"]["rot"]["scaling"].__setitem__("factor", 0), "factor"),
    (lambda c: c["layers"][0]["mlp"]["router"].pop("experts"), "experts"),
    (lambda c: c["layers"][0]["mlp"]["router"].pop("top"), "top"),
    (lambda c: c["layers"][0]["mlp"]["router"].pop("scale"), "scale"),
    (lambda c: c["layers"][0]["mlp"]["router"].__setitem__("identity", -1), "identity"),
    (lambda c: c["layers"][0]["mlp"]["router"]["groups"].__setitem__("count", 4), "groups"),
    (lambda c: c["layers"][0]["mlp"]["router"]["groups"].__setitem__("keep", 4), "groups"),
    (lambda c: c["layers"][0]["mlp"]["router"].__setitem__("top", 5), "5 experts"),
    (lambda c: c["layers"][0]["mlp"].pop("expert"), "ff"),
    (lambda c: c["layers"][0]["mlp"]["shared"].pop("ff"), "ff"),
    (lambda c: c["loop"].__setitem__("stop", 4), "loop"),
    (lambda c: c["loop"].__setitem__("start", 2), "loop"),
    (lambda c: c["loop"].pop("times"), "times"),
])
def test_config_errors_name_the_key(change, word):
    cfg = copy.deepcopy(P.config_a())
    change(cfg)
    with pytest.raises(ConfigError) as e:
        load_model_config(cfg)
    assert word in str(e.value)


@pytest.mark.parametrize("rot", [{"base": 10000.0, "dims": 64, "scaling": {"factor": 4.0, "original": 2048, "fast": 32.0, "slow": 1.0}},
                                 {"base": 500.0, "dims": 8, "scaling": {"factor": 40.0, "original": 64, "fast": 4.0, "slow": 0.01}},
                                 {"base": 7.0, "dims": 4, "scaling": {"factor": 2.0, "original": 100000, "fast": 2.0, "slow": 1.0}},
                                 {"base": 100.0, "dims": 12, "scaling": {"factor": 0.5, "original": 30, "fast": 900.0, "slow": 400.0}}])
def test_stretched_frequencies(rot):
    """The model's frequencies and magnitude are the plain ones; a pair that turns often keeps its rate, one that turns seldom has
    it divided; the upper bound of the ramp is one less than the turned entries, not than the pairs."""
    cfg = P.config_b()
    cfg["layers"][1]["mixer"].update(dim=64, vdim=64, rot=rot)
    arch, c = load_model_config(cfg)
    got = c.layers[1].mixer["rot"]
    want = P.frequencies(rot)
    assert got["frequencies"] == pytest.approx(want, rel=1e-14) and got["magnitude"] == pytest.approx(P.magnitude(rot), rel=1e-14)
    plain = P.frequencies({k: v for k, v in rot.items() if k != "scaling"})
    lo_f, hi_f = sorted((1.0, 1.0 / rot["scaling"]["factor"]))
    assert all(lo_f - 1e-12 <= w / p <= hi_f + 1e-12 for w, p in zip(want, plain))


def test_neutral_values_of_random_weights():
    from infinilm_amd.weights.random_init import random_state_dict
    sd = random_state_dict(P.config_a(), 0, std=0.0, norm_init="one_plus")
    assert sd["l0.norm1.alpha"].shape == () and float(sd["l0.norm1.alpha"]) == 0.5
    assert (sd["l0.norm1"] == 1).all() and (sd["l0.norm1.b"] == 0).all() and (sd["l1.mix.norm"] == 1).all()
    assert (sd["l2.mix.q.norm"] == 1).all() and (sd["l0.mlp.correction"] == 0).all() and (sd["loop.in"] == 0).all()


def test_the_plain_implementation_agrees_with_itself():
    """Logits of a prefix do not depend on what follows; the recurrence without its running maximum (where nothing overflows), as
    sums of weights; groups that are all kept are no groups; a loop of one pass with [I, 0] is no loop."""
    cfg = P.config_a()
    W = P.random_weights(cfg, 1)
    toks = [(7 * i) % 61 for i in range(50)]
    full = P.forward(cfg, W, toks)
    assert torch.allclose(P.forward(cfg, W, toks[:31]), full[:31], atol=1e-10)

    g = torch.Generator().manual_seed(5)
    T, dk, dv = 14, 5, 3
    q, k = (torch.randn((T, dk), generator=g, dtype=torch.float64) for _ in range(2))
    v = torch.randn((T, dv), generator=g, dtype=torch.float64)
    i, f = torch.randn((T,), generator=g, dtype=torch.float64), P.log_sigmoid(torch.randn((T,), generator=g, dtype=torch.float64))
    o = P.mlstm_recurrence(q, k, v, i, f)
    L = torch.cumsum(f, 0)
    for t in range(T):
        wt = torch.exp(L[t] - L[:t + 1] + i[:t + 1])
        m = max(float(L[t]), float((L[t] - L[:t + 1] + i[:t + 1]).max()))
        num, den = (wt * (k[:t + 1] @ q[t])) @ v[:t + 1], float((wt * (k[:t + 1] @ q[t])).sum())
        assert torch.allclose(o[t], num / (max(abs(den), 1.0) + 1e-6 * math.exp(m)), atol=1e-12)

    r = {"experts": 6, "top": 3, "scale": 1.0}
    z, c = torch.randn((6,), generator=g), 0.3 * torch.randn((6,), generator=g)
    assert P.choose(z, c, r).tolist() == P.choose(z, c, dict(r, groups={"count": 3, "keep": 3})).tolist()
    kept = P.choose(z, c, dict(r, top=2, groups={"count": 3, "keep": 1})).tolist()
    assert kept[0] == P.choose(z, c, r).tolist()[0] and kept[0] // 2 == kept[1] // 2

    once, none = P.config_a(), P.config_a()
    once["loop"]["times"] = 1
    none["loop"] = None
    W["loop.in"] = torch.cat([torch.eye(40), torch.zeros((40, 40))], dim=1)
    assert torch.allclose(P.forward(once, W, toks), P.forward(none, W, toks), atol=1e-12)
