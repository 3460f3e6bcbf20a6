"""Zotonex without a GPU: the configuration reader, the tensors the model asks for, its run order with borrowed
caches, what caches read through several chunks keep, and the plain implementation's own special cases."""
import copy

import numpy as np
import pytest

import plain_zotonex as P
from rustinfer_amd.cache import CacheManager
from rustinfer_amd.config import ConfigError, DifferenceAttentionSpec, ZotonexConfig, ZotonexExperts, resolve_architecture
from rustinfer_amd.parts.base import PagedKVNeed

CFG = dict(architecture="Zotonex", vocab=97, width=48, norm=dict(eps=3e-6), embedding=dict(scale=2.5), logit_scale=0.75, layers=[
    dict(type="attention", mixer=dict(heads=6, kv_heads=2, dim=8, vdim=12, scale=0.3, diff=0.4, mask=dict(size=20)),
         mlp=dict(kind="moe", expert=dict(ff=24, limit=1.5), router=dict(experts=5, top=2), shared=dict(ff=40, limit=0.9))),
    dict(type="attention", mixer=dict(heads=1, kv_heads=1, dim=16, vdim=10, scale=0.2, diff=0.1, mask=dict(size=48)), mlp=None),
    dict(type="attention", mixer=dict(heads=6, kv_heads=2, dim=8, vdim=12, scale=0.4, diff=0.2, mask=dict(size=50), kv_from=0),
         mlp=dict(kind="moe", expert=dict(ff=8, limit=2.0), router=dict(experts=3, top=3))),
])


def changed(path, value):
    d = copy.deepcopy(CFG)
    node = d
    for k in path[:-1]:
        node = node[k]
    if value is KeyError:
        del node[path[-1]]
    else:
        node[path[-1]] = value
    return d


def test_reads_every_size_and_constant():
    entry = resolve_architecture(CFG)
    assert entry.name == "Zotonex"
    c = ZotonexConfig.from_dict(CFG)
    assert (c.vocab_size, c.hidden_size, c.norm_eps, c.embedding_scale, c.logit_scale) == (97, 48, 3e-6, 2.5, 0.75)
    assert [x.mixer for x in c.layers] == [DifferenceAttentionSpec(6, 2, 8, 12, 0.3, 0.4, 20), DifferenceAttentionSpec(1, 1, 16, 10, 0.2, 0.1, 48),
                                           DifferenceAttentionSpec(6, 2, 8, 12, 0.4, 0.2, 50, 0)]
    assert [x.mlp for x in c.layers] == [ZotonexExperts(24, 1.5, 5, 2, 40, 0.9), None, ZotonexExperts(8, 2.0, 3, 3)]
    assert ZotonexConfig.from_dict(c.to_dict()) == c


@pytest.mark.parametrize("change,word", [
    ((("layers", 0, "type"), "conv"), "unknown mixer"), ((("layers", 0, "mixer", "kv_heads"), 4), "multiple"),
    ((("layers", 2, "mixer", "kv_from"), 1), "equal"), ((("layers", 2, "mixer", "kv_from"), 2), "kv_from"),
    ((("layers", 2, "mixer", "vdim"), 16), "equal"), ((("layers", 0, "mixer", "mask", "size"), 0), "size"),
    ((("layers", 0, "mixer", "diff"), KeyError), "diff"), ((("layers", 0, "mixer", "dim"), 300), "features"),
    ((("layers", 0, "mlp", "router", "top"), 6), "top"), ((("layers", 0, "mlp", "kind"), "dense"), "kind"),
    ((("layers", 0, "mlp", "expert", "limit"), KeyError), "limit"), ((("layers", 0, "mlp", "shared", "limit"), 0.0), "limit"),
    ((("width",), KeyError), "width"), ((("norm", "eps"), 0.0), "eps")])
def test_refuses_what_it_cannot_run(change, word):
    with pytest.raises(ConfigError) as e:
        ZotonexConfig.from_dict(changed(*change))
    assert word in str(e.value)


def build():
    entry = resolve_architecture(CFG)
    return entry.builder(ZotonexConfig.from_dict(CFG))


def test_model_asks_for_the_designs_tensors():
    W = 48
    want = {"embed": (97, W), "head": (97, W), "final.norm": (W,)}
    for i, (dim, q, o) in enumerate(((8, 96, 72), (16, 32, 10), (8, 96, 72))):
        want.update({f"l{i}.norm1": (W,), f"l{i}.mix.q": (q, W), f"l{i}.mix.q.norm": (dim,), f"l{i}.mix.o": (W, o)})
        want.update({f"l{i}.mix.{n}": (dim,) for n in ("lq1", "lk1", "lq2", "lk2")})
    want.update({"l0.mix.k": (32, W), "l0.mix.v": (24, W), "l0.mix.k.norm": (8,), "l1.mix.k": (32, W), "l1.mix.v": (10, W), "l1.mix.k.norm": (16,)})
    for i, E, F in ((0, 5, 24), (2, 3, 8)):
        want.update({f"l{i}.norm2": (W,), f"l{i}.mlp.router": (E, W)})
        for e in range(E):
            want.update({f"l{i}.mlp.e{e}.gate": (F, W), f"l{i}.mlp.e{e}.up": (F, W), f"l{i}.mlp.e{e}.down": (W, F)})
    want.update({"l0.mlp.shared.gate": (40, W), "l0.mlp.shared.up": (40, W), "l0.mlp.shared.down": (W, 40), "l0.mlp.shared.sg": (1, W)})
    assert {n: tuple(s.shape) for n, s in build().param_specs().items()} == want


def test_run_order_and_what_a_borrowed_cache_must_keep():
    model = build()
    assert [(c.layer, c.cache, c.write) for c in model.schedule] == [(0, 0, True), (1, 1, True), (2, 0, False)]
    assert model.cache_needs() == {0: PagedKVNeed(2, 16, None, 12, 0, (20, 50)), 1: PagedKVNeed(1, 32, None, 10, 0, (48,))}


def test_needs_joined():
    a, w = PagedKVNeed(2, 8, None, 12, 0, (20,)), PagedKVNeed(2, 8, 30, 12, 4)
    assert a.joined(PagedKVNeed(2, 8, None, 12, 0, (7, 20))) == PagedKVNeed(2, 8, None, 12, 0, (7, 20))
    assert a.joined(w) == PagedKVNeed(2, 8, 30, 12, 4, (20,)) and w.joined(PagedKVNeed(2, 8, 40, 12)).window == 40
    assert not a.joined(PagedKVNeed(2, 8, None, 12)).bounded            # a reader of everything keeps everything
    with pytest.raises(ValueError):
        a.joined(PagedKVNeed(2, 8, None, 16, 0, (20,)))
    for need in (a, w, a.joined(w), PagedKVNeed(2, 8, None, None, 0, (20, 50)), PagedKVNeed(2, 8)):
        reach = [need.first_position(p) for p in range(300)]
        assert reach == sorted(reach)                                    # what is out of sight stays out of sight
        for p, lo in enumerate(reach):
            seen = [p // c * c for c in need.chunks] + ([max(0, p + 1 - need.window)] if need.window else [])
            assert lo == (min(seen) if seen else 0)


def test_pages_of_a_chunk_go_back_when_no_layer_reads_them():
    cm = CacheManager(build().cache_needs(), page_size=16, num_pages=12, max_requests=2, max_model_len=192)
    assert [g.need.chunks for g in cm.groups] == [(20, 50), (48,)]
    cm.add_request("a")
    for p in range(150):
        cm.append("a", 1)
        kept = {g.need.chunks: [i for i, page in enumerate(cm.table(g.index, "a")) if page >= 0] for g in cm.groups}
        first = {(20, 50): min(p // 20 * 20, p // 50 * 50), (48,): p // 48 * 48}
        for chunks, pages in kept.items():
            assert pages == list(range(first[chunks] // 16, p // 16 + 1)), (p, chunks)
        cm.check()
    assert cm.pages_held("a") < 2 * 10
    assert cm.can_append([("a", 40)]) and not cm.can_append([("a", 43)])     # (192 positions at most)
    cm.release("a")
    assert cm.free_pages() == 12


def test_plain_mechanisms_reduce_to_known_cases():
    """The oracle itself: one chunk is the causal mask, a chunk of one position returns the position's own value, the
    difference is homogeneous, one expert of score s runs on s h, unclipped limits change nothing."""
    rng = np.random.default_rng(0)
    assert (P.chunk_mask(9, 100) == np.tril(np.ones((9, 9), dtype=bool))).all() and (P.chunk_mask(9, None) == P.chunk_mask(9, 9)).all()
    assert (P.chunk_mask(7, 1) == np.eye(7, dtype=bool)).all()
    assert P.chunk_mask(10, 4).sum(1).tolist() == [1, 2, 3, 4, 1, 2, 3, 4, 1, 2]
    v = rng.standard_normal((6, 5))
    assert np.allclose(P.one_map(rng.standard_normal((6, 3)), rng.standard_normal((6, 3)), v, 0.7, P.chunk_mask(6, 1)), v)
    a, b = rng.standard_normal((2, 6, 8))
    assert np.allclose(P.difference(3 * a, 3 * b, 0.4, 0.25, 1e-30), P.difference(a, b, 0.4, 0.25, 1e-30))
    assert np.allclose(np.mean(P.difference(a, b, 0.4, 0.25, 1e-30) ** 2, axis=1), 0.75 ** 2)
    z = np.zeros(4)
    assert P.map_weight(dict(lq1=z, lk1=z, lq2=z, lk2=z), 0.3) == 0.3
    h = rng.standard_normal((7, 10))
    w = {"router": rng.standard_normal((1, 10)), "e0.gate": rng.standard_normal((6, 10)), "e0.up": rng.standard_normal((6, 10)),
         "e0.down": rng.standard_normal((10, 6))}
    s = P.sigmoid(h @ w["router"].T)
    mlp = dict(kind="moe", expert=dict(ff=6, limit=1e9), router=dict(experts=1, top=1))
    g, u = (s * h) @ w["e0.gate"].T, (s * h) @ w["e0.up"].T
    assert np.allclose(P.routed_ff(h, w, mlp), (g / (1 + np.exp(-1.702 * g)) * (u + 1)) @ w["e0.down"].T)
