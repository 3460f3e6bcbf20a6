"""Sibodra without a GPU: the configuration reader, the tensors the model asks for, its caches, the random-weights mode,
and the plain implementation's own special cases."""
import copy
import math

import numpy as np
import pytest
import torch

import plain_sibodra as P
from rustinfer_amd.config import (CappedAttentionSpec, ConfigError, QueryLatentAttentionSpec, RopeScaling, SibodraConfig,
                                  SibodraFeedForwardSpec, resolve_architecture)
from rustinfer_amd.parts.base import PagedKVNeed

SCALING = dict(factor=3.0, low=1.5, high=5.0, original=100)
CFG = dict(architecture="Sibodra", vocab=97, width=48, streams=3, norm=dict(eps=3e-6), logit_softcap=12.5, layers=[
    dict(type="attention", mixer=dict(heads=6, kv_heads=2, dim=12, vdim=10, scale=0.3, softcap=7.0, rot=dict(base=500.0, dims=8, scaling=SCALING)),
         mlp=dict(kind="moe", expert=dict(ff=24), router=dict(experts=5, top=2), shared=dict(ff=40))),
    dict(type="latent_attention", mixer=dict(heads=3, dim=14, rot_dim=6, vdim=9, q_rank=22, kv_rank=17, scale=0.2, rot=dict(base=900.0, dims=6)), mlp=None),
    dict(type="attention", mixer=dict(heads=1, kv_heads=1, dim=16, vdim=4, scale=0.4, rot=dict(base=70.0, dims=16)), mlp=dict(kind="dense", ff=56)),
    dict(type="latent_attention", mixer=dict(heads=2, dim=4, rot_dim=8, vdim=12, q_rank=10, kv_rank=30, scale=0.1, rot=dict(base=70.0, dims=4, scaling=SCALING)),
         mlp=dict(kind="moe", expert=dict(ff=8), router=dict(experts=3, top=3))),
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
    assert entry.name == "Sibodra"
    c = SibodraConfig.from_dict(CFG)
    assert (c.vocab_size, c.hidden_size, c.streams, c.norm_eps, c.logit_softcap) == (97, 48, 3, 3e-6, 12.5)
    sc = RopeScaling("llama3", 3.0, 1.5, 5.0, 100)
    assert [x.mixer for x in c.layers] == [CappedAttentionSpec(6, 2, 12, 10, 0.3, 7.0, 500.0, 8, sc), QueryLatentAttentionSpec(3, 14, 6, 9, 22, 17, 0.2, 900.0, 6),
                                           CappedAttentionSpec(1, 1, 16, 4, 0.4, None, 70.0, 16), QueryLatentAttentionSpec(2, 4, 8, 12, 10, 30, 0.1, 70.0, 4, sc)]
    assert [x.mlp for x in c.layers] == [SibodraFeedForwardSpec("moe", 24, 5, 2, 40), None, SibodraFeedForwardSpec("dense", 56),
                                         SibodraFeedForwardSpec("moe", 8, 3, 3)]
    assert SibodraConfig.from_dict(c.to_dict()) == c


@pytest.mark.parametrize("change,word", [
    ((("layers", 0, "type"), "conv"), "unknown mixer"), ((("layers", 0, "mixer", "kv_heads"), 4), "multiple"),
    ((("layers", 0, "mixer", "rot", "dims"), 14), "exceeds"), ((("layers", 1, "mixer", "rot", "dims"), 8), "exceeds"),
    ((("layers", 0, "mixer", "rot", "dims"), 7), "even"), ((("layers", 0, "mixer", "rot", "scaling", "high"), 1.0), "high"),
    ((("layers", 0, "mixer", "rot", "scaling", "original"), KeyError), "original"), ((("layers", 0, "mixer", "softcap"), 0.0), "softcap"),
    ((("layers", 0, "mixer", "dim"), 300), "features"), ((("layers", 1, "mixer", "q_rank"), KeyError), "q_rank"),
    ((("layers", 1, "mixer", "kv_rank"), 0), "kv_rank"), ((("layers", 0, "mlp", "router", "top"), 6), "top"),
    ((("layers", 0, "mlp", "kind"), "sparse"), "kind"), ((("layers", 0, "mlp", "shared", "ff"), 0), "ff"),
    ((("width",), KeyError), "width"), ((("streams",), 0), "streams"), ((("streams",), KeyError), "streams"), ((("norm", "eps"), 0.0), "eps"),
    ((("logit_softcap",), -1.0), "softcap")])
def test_refuses_what_it_cannot_run(change, word):
    with pytest.raises(ConfigError) as e:
        SibodraConfig.from_dict(changed(*change))
    assert word in str(e.value)


def build():
    entry = resolve_architecture(CFG)
    return entry.builder(SibodraConfig.from_dict(CFG))


def test_model_asks_for_the_designs_tensors():
    W, n = 48, 3
    want = {"embed": (97, W), "head": (97, W), "final.norm": (W,)}
    for i in range(4):
        want.update({f"l{i}.norm1": (W,), f"l{i}.hc1.in": (n,), f"l{i}.hc1.out": (n,), f"l{i}.hc1.mix": (n, n)})
        if i != 1:
            want.update({f"l{i}.norm2": (W,), f"l{i}.hc2.in": (n,), f"l{i}.hc2.out": (n,), f"l{i}.hc2.mix": (n, n)})
    for i, H, G, d, dv in ((0, 6, 2, 12, 10), (2, 1, 1, 16, 4)):
        want.update({f"l{i}.mix.q": (H * d, W), f"l{i}.mix.k": (G * d, W), f"l{i}.mix.v": (G * dv, W), f"l{i}.mix.q.norm": (d,),
                     f"l{i}.mix.k.norm": (d,), f"l{i}.mix.g": (H, W), f"l{i}.mix.o": (W, H * dv)})
    for i, H, d, r, dv, Q, R in ((1, 3, 14, 6, 9, 22, 17), (3, 2, 4, 8, 12, 10, 30)):
        want.update({f"l{i}.mix.dq": (Q, W), f"l{i}.mix.dq.norm": (Q,), f"l{i}.mix.uq": (H * (d + r), Q), f"l{i}.mix.dkv": (R + r, W),
                     f"l{i}.mix.dkv.norm": (R,), f"l{i}.mix.uk": (H * d, R), f"l{i}.mix.uv": (H * dv, R), f"l{i}.mix.g": (H * dv, W),
                     f"l{i}.mix.o": (W, H * dv)})
    for i, E, F in ((0, 5, 24), (3, 3, 8)):
        want.update({f"l{i}.mlp.router": (E, W), f"l{i}.mlp.router.b": (E,)})
        for e in range(E):
            want.update({f"l{i}.mlp.e{e}.up": (F, W), f"l{i}.mlp.e{e}.down": (W, F)})
    want.update({"l0.mlp.shared.up": (40, W), "l0.mlp.shared.down": (W, 40)})
    want.update({"l2.mlp.gate": (56, W), "l2.mlp.up": (56, W), "l2.mlp.down": (W, 56)})
    assert {k: tuple(s.shape) for k, s in build().param_specs().items()} == want


def test_run_order_and_caches():
    model = build()
    assert [(c.layer, c.cache, c.write) for c in model.schedule] == [(i, i, True) for i in range(4)]
    assert model.cache_needs() == {0: PagedKVNeed(2, 12, None, 10), 1: PagedKVNeed(1, 23, None, 17), 2: PagedKVNeed(1, 16, None, 4), 3: PagedKVNeed(1, 38, None, 30)}
    assert model.graph_safe


def test_a_random_model_can_be_written_and_read(tmp_path):
    from rustinfer_amd.weights import write_random_model
    write_random_model(SibodraConfig.from_dict(CFG), 3, str(tmp_path))
    cfg, w = P.read_model(str(tmp_path))
    assert SibodraConfig.from_dict(cfg) == SibodraConfig.from_dict(CFG)
    logits = P.forward(cfg, w, [5, 96, 0, 41])
    assert logits.shape == (4, 97) and np.isfinite(logits).all() and np.abs(logits).max() < 12.5
    assert np.abs(w["l0.hc1.mix"] - np.eye(3)).max() < 1.0 and abs(w["l0.hc1.in"].sum() - 1.0) < 1.0


def test_rotation_tables_are_the_plain_frequencies():
    from rustinfer_amd.parts import rotary_frequencies
    for dims, base, sc in ((8, 500.0, SCALING), (64, 10000.0, dict(factor=8.0, low=1.0, high=4.0, original=50)), (16, 70.0, None),
                           (32, 2000.0, dict(factor=40.0, low=1.0, high=32.0, original=300))):
        s = RopeScaling("llama3", sc["factor"], sc["low"], sc["high"], sc["original"]) if sc else None
        want = P.frequencies(dict(base=base, dims=dims, scaling=sc))
        assert np.allclose(rotary_frequencies(dims, base, s).numpy(), want, rtol=1e-12)
        if sc:                                         # all three bands are there
            plain = P.frequencies(dict(base=base, dims=dims))
            ratio = plain / want
            assert ratio.min() == 1.0 and abs(ratio.max() - sc["factor"]) < 1e-9


def test_plain_mechanisms_reduce_to_known_cases():
    """The oracle itself: one stream with unit weights is the residual sum, an added one is a key of score 0 with value 0, a
    wide cap changes nothing, the chosen softmax over all experts is the softmax, a score's cap bounds it."""
    rng = np.random.default_rng(0)
    X, y = rng.standard_normal((5, 1, 7)), rng.standard_normal((5, 7))
    assert np.allclose(P.write_streams(X, np.eye(1), np.ones(1), y)[:, 0], X[:, 0] + y)
    M = rng.standard_normal((3, 3))
    X3 = rng.standard_normal((5, 3, 7))
    assert np.allclose(P.write_streams(X3, M, np.zeros(3), y), np.einsum("st,psd->ptd", M, X3))       # from, to
    assert np.allclose(P.read_streams(X3, np.array([0.0, 1.0, 0.0])), X3[:, 1])
    q, k, v = rng.standard_normal((6, 4)), rng.standard_normal((6, 4)), rng.standard_normal((6, 3))
    a = P.softmax_attention(q, k, v, 0.7, one_more=True)
    k0, v0 = np.concatenate([np.zeros((1, 4)), k]), np.concatenate([np.zeros((1, 3)), v])
    b = P.softmax_attention(np.concatenate([np.zeros((1, 4)), q]), k0, v0, 0.7)[1:]
    assert np.allclose(a, b)
    assert np.allclose(P.softmax_attention(q, k, v, 0.7, cap=1e7), P.softmax_attention(q, k, v, 0.7), atol=1e-6)
    assert np.abs(P.softcap(1e3 * rng.standard_normal(50), 5.0)).max() <= 5.0
    z = rng.standard_normal(6)
    idx, p = P.chosen_weights(z, 6)
    assert np.allclose(p[np.argsort(idx)], np.exp(z) / np.exp(z).sum())
    w = rng.standard_normal(9)
    x = rng.standard_normal((4, 9)) + 30.0
    n = torch.nn.functional.layer_norm(torch.tensor(x), (9,), torch.tensor(w), None, 1e-5).numpy()
    assert np.allclose(P.layer_norm(x, w, 1e-5), n)
    assert np.allclose(P.rotate(np.ones((3, 2)), dict(base=10.0, dims=2))[2], [math.cos(2) - math.sin(2), math.cos(2) + math.sin(2)])
