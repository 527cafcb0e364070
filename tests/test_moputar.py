"""Moputar without a GPU: config.json's keys and their errors, the tensor names against the plain list, the cache entries a
model asks for (a reader of another layer's keys, chunks of both), the pages that chunks of positions hold and give back, the
random weights' neutral values, and the plain implementation's own consistency."""
import copy

import pytest
import torch

import plain_moputar as P
from infinilm_amd.cache import CacheManager, FixedState, PagedKV
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
    assert spec.architecture == "Moputar" and spec.streams == cfg["streams"]


def test_cache_entries_of_readers_and_writers():
    spec, model = _build(P.config_a())
    assert [(r.layer, r.cache, r.borrows) for r in spec.order] == [(0, 0, None), (1, 1, None), (2, 2, 0), (3, 3, None)]
    # the writer's pages serve chunks of 20 (its own) and of 33 (the reader's); the reader has its convolution's inputs alone
    assert model.cache_needs[0] == (PagedKV(2, 32, chunks=(20, 33)), FixedState((2, 4 * 12 + 2 * 12 + 2 * 20), torch.float32))
    assert model.cache_needs[2] == FixedState((1, 4 * 12), torch.float32)
    assert model.cache_needs[1] == (FixedState((1, 2 * 2 * 10 + 6 * 14), torch.float32), FixedState((6, 14, 10), torch.float32))
    assert model.blocks[0].mixer.chunk == 20 and model.blocks[2].mixer.chunk == 33
    # a writer without a mask keeps everything, whatever its reader sees; a reader without a convolution has no entry
    spec, model = _build(P.config_b())
    assert model.cache_needs[1] == PagedKV(3, 16)
    assert [(r.cache, r.borrows) for r in spec.order] == [(0, None), (1, None), (None, 1), (2, None), (3, None)]
    assert model.blocks[2].mixer.chunk == 50 and model.blocks[2].mixer.cache_chunks == ()


def test_what_config_leaves_out_does_not_exist():
    _, model = _build(P.config_b())
    m = model.blocks[1].mixer
    assert m.taps == 0 and m.rd == 0 and m.chunk == 0 and m.window == 0
    assert model.blocks[1].ffn is None and model.blocks[0].ffn is not None
    cfg = P.config_b()
    del cfg["layers"][0]["mixer"]["conv"]
    _, model = _build(cfg)
    assert model.blocks[0].mixer.taps == 0
    assert {k: tuple(p.shape) for k, p in model.named_parameters().items()} == P.tensor_shapes(cfg)


@pytest.mark.parametrize("change,word", [
    (lambda c: c.pop("width"), "width"),
    (lambda c: c.pop("streams"), "streams"),
    (lambda c: c.__setitem__("streams", 0), "streams"),
    (lambda c: c["norm"].pop("eps"), "eps"),
    (lambda c: c.__setitem__("layers", []), "layers"),
    (lambda c: c["layers"][0].__setitem__("type", "retention"), "retention"),
    (lambda c: c["layers"][0]["mixer"].__setitem__("heads", 3), "heads"),
    (lambda c: c["layers"][1]["mixer"].__setitem__("kv_heads", 4), "kv_heads"),
    (lambda c: c["layers"][0]["mixer"].pop("scale"), "scale"),
    (lambda c: c["layers"][0]["mixer"]["rot"].__setitem__("dims", 5), "dims"),
    (lambda c: c["layers"][0]["mixer"]["rot"].__setitem__("dims", 14), "dims"),
    (lambda c: c["layers"][0]["mixer"]["rot"].pop("base"), "base"),
    (lambda c: c["layers"][0]["mixer"]["mask"].__setitem__("size", 0), "size"),
    (lambda c: c["layers"][2]["mixer"].__setitem__("kv_from", 2), "kv_from"),
    (lambda c: c["layers"][2]["mixer"].__setitem__("kv_from", 1), "kv_from"),
    (lambda c: c["layers"][2]["mixer"].__setitem__("dim", 16), "dim"),
    (lambda c: c["layers"][1]["mixer"].pop("vdim"), "vdim"),
    (lambda c: c["layers"][0]["mlp"].__setitem__("kind", "moe"), "moe"),
    (lambda c: c["layers"][0]["mlp"].pop("ff"), "ff"),
])
def test_config_errors_name_the_key(change, word):
    cfg = copy.deepcopy(P.config_a())
    change(cfg)
    with pytest.raises(ConfigError) as e:
        load_model_config(cfg)
    assert word in str(e.value)


def test_pages_of_chunks_are_given_back():
    """Chunks of 20 and 33 positions on pages of 4: the pages before the earlier of the two chunks' starts go back, the others
    stay; a group of plain windows and one that keeps all are beside it."""
    cm = CacheManager([PagedKV(1, 16, chunks=(20, 33)), PagedKV(1, 16), PagedKV(1, 16, chunks=(20,)), PagedKV(1, 16, chunks=(33, 20))],
                      page_size=4, num_pages=60, max_requests=2, dtype=torch.float32, device="cpu", prefix_caching=True)
    assert len(cm.groups) == 3 and not cm.prefix_caching
    assert [(g.keeps_all, g.span) for g in cm.groups] == [(False, 33), (True, 0), (False, 20)]
    cm.admit("a")
    for n in (19, 1, 1, 12, 7, 26, 1, 30):
        cm.reserve("a", n)
        cm.commit("a", n)
        length = cm.length("a")
        for g, sizes in ((0, (20, 33)), (1, ()), (2, (20,))):
            first = min((length - length % s for s in sizes), default=0) // 4
            table = cm.table("a", g)
            assert all(p < 0 for p in table[:first]) and all(p >= 0 for p in table[first:]), (length, g)
        cm.check()
    cm.release("a")
    assert all(cm.free_pages(g) == 60 for g in range(3))
    with pytest.raises(ValueError):
        PagedKV(1, 16, window=8, chunks=(4,))


def test_scheduler_counts_chunks_as_windows():
    from infinilm_amd.engine.scheduler import Scheduler
    cm = CacheManager([PagedKV(1, 16, chunks=(64,))], page_size=16, num_pages=8, max_requests=2, dtype=torch.float32, device="cpu")
    s = Scheduler.__new__(Scheduler)
    s.cache, s.chunk_size, s.max_num_batched_tokens = cm, 32, 100
    assert s._group_pages(cm.groups[0], 10 ** 6) == 4 + 2 + 1
    assert s._group_pages(cm.groups[0], 30) == 2


def test_neutral_values_of_random_weights():
    from infinilm_amd.weights.random_init import random_state_dict
    sd = random_state_dict(P.config_a(), 0, std=0.0, norm_init="one_plus")
    assert torch.equal(sd["l0.hc1.mix"], torch.eye(3)) and torch.allclose(sd["l0.hc1.in"], torch.full((3,), 1 / 3))
    assert (sd["l0.hc2.out"] == 1).all() and (sd["l0.norm1"] == 0).all() and (sd["final.norm"] == 0).all()
    assert (sd["l0.mix.q.norm"] == 1).all() and (sd["l1.mix.norm"] == 1).all() and (sd["l1.mix.q"] == 0).all()


def test_the_plain_implementation_agrees_with_itself():
    """Logits of a prefix do not depend on what follows; chunks longer than the sequence are no chunks; the recurrence written as
    products of matrices over the whole sequence; streams that start equal and mix by the identity are one stream."""
    cfg = P.config_a()
    W = P.random_weights(cfg, 1)
    toks = list(range(70))
    full = P.forward(cfg, W, toks)
    assert torch.allclose(P.forward(cfg, W, toks[:41]), full[:41], atol=1e-10)
    wide, none = copy.deepcopy(cfg), copy.deepcopy(cfg)
    for i in (0, 2):
        wide["layers"][i]["mixer"]["mask"] = {"size": 70}
        del none["layers"][i]["mixer"]["mask"]
    a, b = P.forward(wide, W, toks), P.forward(none, W, toks)
    assert torch.allclose(a, b, atol=1e-12) and not torch.allclose(a, full, atol=1e-6)
    assert P.visible(7, 3)[4].tolist() == [False, False, False, True, True, False, False]

    g = torch.Generator().manual_seed(5)
    T, H, dk, dv = 12, 2, 5, 3
    q, k = (torch.nn.functional.normalize(torch.randn((T, H, dk), generator=g, dtype=torch.float64), dim=-1) for _ in range(2))
    v = torch.randn((T, H, dv), generator=g, dtype=torch.float64)
    dec, beta = torch.rand((T, H), generator=g, dtype=torch.float64), torch.rand((T, H), generator=g, dtype=torch.float64)
    o, S = P.delta_rule(q, k, v, dec, beta)
    for h in range(H):
        M = torch.zeros((dk, dv), dtype=torch.float64)
        for t in range(T):      # S <- g (I - beta k k^T) S + beta k v^T
            K = k[t, h][:, None]
            M = dec[t, h] * (M - beta[t, h] * K @ (K.T @ M)) + beta[t, h] * K @ v[t, h][None]
            assert torch.allclose(M.T @ q[t, h], o[t, h], atol=1e-12)
        assert torch.allclose(M, S[h], atol=1e-12)

    one = dict(cfg, streams=1)
    W1 = P.random_weights(one, 1)
    three = {k: v for k, v in W1.items()}
    for i in range(4):
        for q in (1, 2):
            if f"l{i}.hc{q}.in" in W1:
                W1[f"l{i}.hc{q}.mix"] = torch.ones((1, 1))
                three[f"l{i}.hc{q}.in"] = W1[f"l{i}.hc{q}.in"].repeat(3) / 3
                three[f"l{i}.hc{q}.out"], three[f"l{i}.hc{q}.mix"] = W1[f"l{i}.hc{q}.out"].repeat(3), torch.eye(3)
    # the final norm takes the streams' sum: three times the row, which its division takes out but for eps
    assert torch.allclose(P.forward(cfg, three, toks), P.forward(one, W1, toks), atol=1e-4)
