"""Zotonex on the GPU against the plain implementation (``plain_zotonex.py``): every mechanism alone, then whole
models of three small configurations that differ in every size, in their chunks and in which layers borrow keys and
values, through every way of cutting requests into steps, through pages and slots that are used again, and through
``LLM.generate``.  Weights are drawn here with deviations that make activations of order one; a few tests build
inputs so that one key at a chunk's edge decides, and plant a mistake in the plain implementation to see that they
could tell."""
import json
import math
import os

import numpy as np
import pytest
import torch

import plain_zotonex as P
from helpers import cut_mixed, cut_portions, cut_tail_single, cut_whole, random_requests, run_steps
from test_gpu_belorax import CUTS, PART_TOL, Rows, check_rows, portion_kernel, rel, run_part, some_rows  # noqa: F401

pytestmark = pytest.mark.gpu
DEV = "cuda:0"


def att(heads, kv, dim, vdim, scale, size, diff=0.3, kv_from=None):
    m = dict(heads=heads, kv_heads=kv, dim=dim, vdim=vdim, scale=scale, diff=diff)
    if size is not None:
        m["mask"] = dict(size=size)
    if kv_from is not None:
        m["kv_from"] = kv_from
    return m


def moe(experts, top, ff, limit, shared_ff, shared_limit):
    d = dict(kind="moe", expert=dict(ff=ff, limit=limit), router=dict(experts=experts, top=top))
    if shared_ff:
        d["shared"] = dict(ff=shared_ff, limit=shared_limit)
    return d


def layer(mixer, mlp):
    return dict(type="attention", mixer=mixer, mlp=mlp)


CONFIGS = {
    # chunks of no round size, a borrower with longer chunks than the cache's owner, a layer without feed-forward
    "A": dict(architecture="Zotonex", vocab=200, width=72, norm=dict(eps=1e-5), embedding=dict(scale=3.0), logit_scale=0.5, layers=[
        layer(att(4, 2, 12, 20, 0.3, 20, 0.2), moe(5, 2, 24, 0.8, 40, 1.1)),
        layer(att(4, 2, 12, 20, 0.35, 33, 0.5, kv_from=0), moe(4, 1, 16, 2.0, 8, 0.6)),
        layer(att(2, 1, 24, 16, 0.2, 11, 0.7), None),
        layer(att(4, 2, 12, 20, 0.25, 9, 0.1, kv_from=0), moe(3, 3, 12, 0.5, 24, 3.0)),
    ]),
    # heads beyond one 64-wide slice, chunks at page borders, more experts than a wave has lanes, borrowers far behind
    "B": dict(architecture="Zotonex", vocab=333, width=136, norm=dict(eps=1e-6), embedding=dict(scale=1.0), logit_scale=1.0, layers=[
        layer(att(8, 2, 40, 132, 0.15, 64, 0.4), moe(70, 3, 16, 1.5, 56, 1.0)),
        layer(att(3, 3, 72, 40, 0.11, 48, 0.3), moe(9, 4, 32, 0.7, 32, 0.7)),
        layer(att(8, 2, 40, 132, 0.12, 64, 0.6, kv_from=0), None),
        layer(att(3, 3, 72, 40, 0.1, None, 0.2, kv_from=1), moe(6, 1, 48, 1.0, 0, 0.0)),
        layer(att(8, 2, 40, 132, 0.17, 32, 0.25, kv_from=0), moe(2, 2, 40, 5.0, 16, 0.4)),
    ]),
    # a width and a vocabulary that are no multiples of eight, odd head sizes, three query heads a key/value head
    "C": dict(architecture="Zotonex", vocab=211, width=100, norm=dict(eps=1e-6), embedding=dict(scale=0.5), logit_scale=2.0, layers=[
        layer(att(3, 1, 6, 10, 0.5, 7, 0.8), moe(5, 2, 12, 1.2, 20, 0.9)),
        layer(att(3, 1, 6, 10, 0.4, 7, 0.3, kv_from=0), moe(8, 3, 10, 0.6, 6, 2.0)),
        layer(att(5, 5, 18, 14, 0.3, 50, 0.0), moe(4, 2, 30, 1.0, 12, 1.0)),
        layer(att(16, 1, 8, 12, 0.35, 17, 0.45), moe(7, 1, 9, 0.9, 33, 0.8)),
    ]),
}
PAGE = {"A": 8, "B": 16, "C": 16}


def bf16_round(a: np.ndarray) -> torch.Tensor:
    return torch.tensor(a, dtype=torch.float32).to(torch.bfloat16)


def draw_weights(cfg: dict, seed: int):
    """name -> bfloat16 tensor for every tensor of the design, activations of order one, limits that clip."""
    rng = np.random.default_rng(seed)
    W = cfg["width"]
    mat = lambda o, i, s=1.0: bf16_round(s * rng.standard_normal((o, i)) / math.sqrt(i))
    vec = lambda n, mean, std: bf16_round(mean + std * rng.standard_normal(n))
    t = {"embed": bf16_round(rng.standard_normal((cfg["vocab"], W))), "final.norm": vec(W, 1.0, 0.2), "head": mat(cfg["vocab"], W)}
    for i, lay in enumerate(cfg["layers"]):
        m, p, mlp = lay["mixer"], f"l{i}.", lay["mlp"]
        t[p + "norm1"] = vec(W, 1.0, 0.2)
        t[p + "mix.q"], t[p + "mix.q.norm"] = mat(m["heads"] * 2 * m["dim"], W), vec(m["dim"], 1.5, 0.3)
        if m.get("kv_from") is None:
            t[p + "mix.k"], t[p + "mix.k.norm"] = mat(m["kv_heads"] * 2 * m["dim"], W), vec(m["dim"], 1.5, 0.3)
            t[p + "mix.v"] = mat(m["kv_heads"] * m["vdim"], W)
        for n in ("lq1", "lk1", "lq2", "lk2"):
            t[p + "mix." + n] = vec(m["dim"], 0.0, 0.2)
        t[p + "mix.o"] = mat(W, m["heads"] * m["vdim"])
        if mlp is None:
            continue
        F = mlp["expert"]["ff"]
        t[p + "norm2"] = vec(W, 1.0, 0.2)
        t[p + "mlp.router"] = mat(mlp["router"]["experts"], W, 3.0)
        for e in range(mlp["router"]["experts"]):
            t[p + f"mlp.e{e}.gate"], t[p + f"mlp.e{e}.up"], t[p + f"mlp.e{e}.down"] = mat(F, W, 2.0), mat(F, W, 2.0), mat(W, F)
        if mlp.get("shared"):
            S = mlp["shared"]["ff"]
            t[p + "mlp.shared.gate"], t[p + "mlp.shared.up"], t[p + "mlp.shared.down"] = mat(S, W, 2.0), mat(S, W, 2.0), mat(W, S)
            t[p + "mlp.shared.sg"] = mat(1, W, 2.0)
    return t


@pytest.fixture(scope="module")
def tdirs(tmp_path_factory):
    from rustinfer_amd.weights import write_safetensors
    out = {}
    for k, (name, cfg) in enumerate(CONFIGS.items()):
        d = str(tmp_path_factory.mktemp("zotonex_" + name))
        with open(os.path.join(d, "config.json"), "w") as f:
            json.dump(cfg, f)
        write_safetensors(os.path.join(d, "model.safetensors"), draw_weights(cfg, 51 + k))
        out[name] = d
    return out


@pytest.fixture(scope="module")
def plain(tdirs):
    return {name: P.read_model(d) for name, d in tdirs.items()}


def plain_rows(cfg, w, reqs):
    rows = Rows()
    rows.margin = {}
    for rid, toks in reqs.items():
        gaps = []
        rows[rid] = P.forward(cfg, w, toks, gaps=gaps)
        rows.margin[rid] = np.min(np.stack(gaps), axis=0) / 2.0 if gaps else np.full(len(toks), np.inf)
    return rows


@pytest.fixture(scope="module")
def plain_logits(plain):
    memo = {}

    def get(name, lengths, seed):
        key = (name, tuple(lengths), seed)
        if key not in memo:
            cfg, w = plain[name]
            reqs = random_requests(cfg["vocab"], lengths, seed)
            memo[key] = (reqs, plain_rows(cfg, w, reqs))
        return memo[key]
    return get


def engine_for(model_dir, dtype, name, num_pages=64, max_requests=4, max_len=512):
    from rustinfer_amd.engine import build_engine
    return build_engine(model_dir, dtype=dtype, device=DEV, page_size=PAGE[name], num_pages=num_pages,
                        max_requests=max_requests, max_model_len=max_len, max_batch_tokens=2048)


# ---------------------------------------------------------------------------
# each mechanism alone
# ---------------------------------------------------------------------------
def attention_part(width, m, eps=1e-5):
    from rustinfer_amd.parts import WindowAttention
    return WindowAttention(width, m["heads"], m["kv_heads"], m["dim"], m["vdim"], m["scale"], qk_norm_eps=eps,
                           chunk=m["mask"]["size"] if m.get("mask") else None, difference=m["diff"], difference_eps=eps)


def load_part(part, seed, dtype, scale=1.0, replace=()):
    """Random weights into ``part``; returns them as the plain implementation reads them."""
    from rustinfer_amd.engine import make_runtime
    g = torch.Generator().manual_seed(seed)
    wt = {}
    for n, s in part.param_specs().items():
        if len(s.shape) == 2:
            wt[n] = (torch.randn(s.shape, generator=g) * scale / math.sqrt(s.shape[1])).to(torch.bfloat16)
        elif n.endswith("norm"):
            wt[n] = (1.0 + torch.randn(s.shape, generator=g) * 0.2).to(torch.bfloat16)
        else:
            wt[n] = (torch.randn(s.shape, generator=g) * 0.3).to(torch.bfloat16)
    for n, t in dict(replace).items():
        assert n in wt and tuple(wt[n].shape) == tuple(t.shape)
        wt[n] = t.to(torch.bfloat16)
    part.load(wt, make_runtime(dtype, DEV))
    return {n: t.double().numpy() for n, t in wt.items()}


def plain_attention(xs, w, m, eps=1e-5):
    return P.attention(xs, w, m, eps, P.keys_values(xs, w, m, eps))


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("H,G,dk,dv,scale,size,diff", [
    (4, 2, 16, 24, 0.3, 23, 0.3), (3, 3, 40, 36, 0.2, 64, 0.0), (8, 1, 32, 16, 0.18, 16, 0.8), (2, 2, 128, 128, 0.09, 100, 0.5),
    (5, 5, 72, 200, 0.12, 7, 0.1), (6, 1, 24, 40, 0.2, 150, 0.6), (2, 1, 256, 256, 0.06, 40, 0.4), (1, 1, 6, 2, 0.5, 1, 0.2),
    (16, 1, 8, 12, 0.35, 48, 0.45), (6, 2, 64, 128, 0.12, None, 0.3), (12, 4, 24, 72, 0.25, 33, 0.9), (3, 1, 10, 100, 0.3, 5, 0.35),
    (10, 1, 16, 64, 0.3, 80, 0.25), (4, 4, 104, 256, 0.1, 33, 0.3), (9, 3, 40, 56, 0.2, None, 0.15)])
def test_difference_attention_alone(dtype, H, G, dk, dv, scale, size, diff, portion_kernel):
    d, m = 48, att(H, G, dk, dv, scale, size, diff)
    part = attention_part(d, m)
    w = load_part(part, H * dk + dv, dtype, scale=2.0)
    x = some_rows(sum(CUTS), d, 5)
    ref = plain_attention(x.double().numpy(), w, m)
    page = 16 if portion_kernel == "parts" else 8
    assert rel(run_part(part, [], dtype, x, CUTS, page=page), ref) < PART_TOL[dtype]
    other = some_rows(60, d, 8)
    assert rel(run_part(part, [], dtype, x, CUTS, page=page, batch_with=other), ref) < PART_TOL[dtype]     # another request beside it


@pytest.mark.parametrize("size", [None, 4100])
def test_thousands_of_keys(size):
    """A prompt of 4,300 tokens and single tokens behind it: more stretches of keys than a row may leave partial
    results of, so that a wave of the single-token kernel takes several; every query has a favourite far back."""
    T, d = 4330, 32
    m = att(4, 2, 16, 24, 1.2, size, 0.3)
    part = attention_part(d, m)
    w = load_part(part, 3, "bfloat16", scale=2.0)
    x = some_rows(T, d, 11)
    ref = plain_attention(x.double().numpy(), w, m)
    cuts = [2048, 2200, 52] + [1] * 30
    got = run_part(part, [], "bfloat16", x, cuts, page=16, num_pages=300, max_len=4400)
    assert rel(got[:4100], ref[:4100]) < PART_TOL["bfloat16"] and rel(got[4100:], ref[4100:]) < PART_TOL["bfloat16"]


def test_weights_keep_their_32_bits(monkeypatch):
    """The bfloat16 kernels against the 32-bit ones on the same bfloat16 queries, keys and values: far closer than
    weights rounded to bfloat16 would be (4e-3), in portions and in single tokens."""
    from rustinfer_amd.kernels import ops
    d, m = 48, att(4, 2, 64, 64, 0.12, 100, 0.3)
    x = some_rows(sum(CUTS), d, 5)
    outs = []
    for parts in (True, False):
        monkeypatch.setattr(ops, "WINDOW_ATTENTION_PARTS", parts)
        keep = []
        real = ops.window_attention

        def both(q, out, *args, **kw):
            wide = torch.empty(out.shape, device=out.device, dtype=torch.bfloat16)
            real(q, wide, *args, **kw)
            out.copy_(wide)
            keep.append(wide.double().cpu().numpy())
        monkeypatch.setattr(ops, "window_attention", both)
        part = attention_part(d, m)
        load_part(part, 5, "bfloat16", scale=2.0)
        run_part(part, [], "bfloat16", x, CUTS, page=16)
        monkeypatch.setattr(ops, "window_attention", real)
        outs.append(np.concatenate(keep))
    diff = np.abs(outs[0] - outs[1])
    # results that round to neighbouring bfloat16 numbers now and then, almost never further apart
    assert (diff > 0).mean() < 0.02 and diff.max() < 2.0 ** -7 * np.abs(outs[1]).max()


@pytest.mark.parametrize("mistake", ["maps swapped", "values of the second map", "no second map", "no factor", "one less in the exponent"])
def test_the_attention_test_could_tell(mistake, monkeypatch):
    """Mistakes planted in the plain implementation move its result far beyond the tolerances above."""
    d, m = 48, att(4, 2, 16, 24, 0.3, 23, 0.3)
    part = attention_part(d, m)
    g = torch.Generator().manual_seed(1)
    w = {n: torch.randn(s.shape, generator=g).double().numpy() * (2.0 / math.sqrt(d) if len(s.shape) == 2 else 0.3)
         for n, s in part.param_specs().items()}
    w["q.norm"], w["k.norm"] = 1.0 + w["q.norm"], 1.0 + w["k.norm"]
    x = some_rows(80, d, 5).double().numpy()
    ref = plain_attention(x, w, m)
    if mistake == "maps swapped":
        keep = P.difference
        monkeypatch.setattr(P, "difference", lambda a, b, *rest: keep(b, a, *rest))
    elif mistake == "values of the second map":
        monkeypatch.setattr(P, "difference", lambda a, b, lam, diff, eps: P.unit(a - b, eps) * (1.0 - diff))
    elif mistake == "no second map":
        monkeypatch.setattr(P, "map_weight", lambda w_, diff: 0.0)
    elif mistake == "no factor":
        monkeypatch.setattr(P, "difference", lambda a, b, lam, diff, eps: P.unit(a - lam * b, eps))
    else:
        monkeypatch.setattr(P, "map_weight", lambda w_, diff: float(np.exp(np.sum(w_["lq1"] * w_["lk1"])) - np.exp(np.sum(w_["lq2"] * w_["lk2"]))))
    assert rel(plain_attention(x, w, m), ref) > 2 * PART_TOL["bfloat16"]


def test_two_maps_that_agree_leave_only_the_eps():
    """Equal maps and a weight of one: the difference is zero, and zero divided by sqrt(eps) is zero."""
    d, m = 32, att(2, 1, 8, 16, 0.3, 20, 1e-9)
    part = attention_part(d, m)
    g = torch.Generator().manual_seed(3)
    q, k = torch.randn(2, 1, 8, d, generator=g), torch.randn(1, 1, 8, d, generator=g)
    zero = torch.zeros(8)
    load_part(part, 9, "float32", replace={"q": q.expand(2, 2, 8, d).reshape(32, d), "k": k.expand(1, 2, 8, d).reshape(16, d),
                                           "lq1": zero, "lk1": zero, "lq2": zero - 40.0, "lk2": zero + 40.0})
    assert abs(part.lam - 1.0) < 1e-6
    got = run_part(part, [], "float32", some_rows(sum(CUTS), d, 4), CUTS)
    assert np.abs(got).max() < 1e-2


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("decoded", [False, True])
@pytest.mark.parametrize("which", [0, 1])
@pytest.mark.parametrize("size", [48, 100, 128, 141])
def test_keys_at_the_edges_of_a_chunk_decide(dtype, decoded, which, size, portion_kernel, monkeypatch):
    """Queries that match one key each in one of the two maps (the other map's query is zero: it weighs all keys
    alike): a chunk's first key is seen from the chunk and not from the next one; the key just before a
    chunk is not seen from it; nor is the first key of the chunk before by a chunk's first query.  A chunk's border that is
    one position off changes these rows beyond any rounding."""
    T, dk, dv = 480, 16, 12
    c0 = -(-300 // size) * size                            # a chunk's first position
    pairs = {c0 - 1: c0 - size, c0: c0 - 1, c0 + 3: c0, c0 + 7: c0 - 1, c0 + 11: c0 + 2, c0 + 17: c0 - size, c0 + 30: (c0 + 15) // 16 * 16}
    g = torch.Generator().manual_seed(2)
    features = {k: n for n, k in enumerate(sorted(set(pairs.values())))}
    assert len(features) <= 6 and max(pairs) < T
    look, eye = torch.zeros(dk, dk), torch.eye(dk)          # a query reads feature 8 + n into key feature n
    x = 0.05 * torch.randn(T, dk, generator=g)
    x[:, 8:] = 0.0
    x[:, 14] = 1.0
    for kpos, n in features.items():
        look[n, 8 + n] = 1.0
        x[kpos, :8] = 0.0
        x[kpos, n] = 4.0
    for qpos, kpos in pairs.items():
        x[qpos, 8 + features[kpos]] = 4.0
    x = x.to(torch.bfloat16).float()
    m = att(1, 1, dk, dv, 1.0, size, 0.4)
    part = attention_part(dk, m, eps=1e-6)
    zero = torch.zeros(dk, dk)
    maps = [look, zero] if which == 0 else [zero, look]
    w = load_part(part, 5, dtype, replace={"q": torch.cat(maps), "k": torch.cat([eye, eye]), "q.norm": torch.ones(dk), "k.norm": torch.ones(dk)})
    xs = x.double().numpy()
    ref = plain_attention(xs, w, m, 1e-6)
    size_right = np.abs(ref).max()
    with monkeypatch.context() as mp:
        for shift in (-1, 1):
            mp.setattr(P, "chunk_mask", lambda n, s, _d=shift: (np.arange(n)[None, :] <= np.arange(n)[:, None])
                       & ((np.arange(n)[:, None] + _d) // s == (np.arange(n)[None, :] + _d) // s))
            off = plain_attention(xs, w, m, 1e-6)
            changed = [q for q in pairs if np.abs(ref[q] - off[q]).max() > 0.2 * size_right]
            assert changed, shift                           # the test can tell
    cuts = [290] + [1] * 190 if decoded else [290, 17, 50, 2, 61, 40, 20]
    got = run_part(part, [], dtype, x, cuts, page=16)
    for qpos in pairs:
        assert np.abs(got[qpos] - ref[qpos]).max() < PART_TOL[dtype] * size_right, qpos


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("E,top,F,limit,S,slimit,rows", [
    (4, 1, 24, 0.7, 40, 1.3, 70), (16, 3, 56, 1.0, 8, 0.4, 5), (70, 3, 16, 2.0, 33, 1.0, 100), (6, 6, 8, 0.3, 24, 0.3, 33),
    (3, 2, 41, 1.0, 0, 0.0, 1), (130, 8, 4, 0.9, 12, 7.0, 17), (1, 1, 32, 0.8, 16, 0.8, 65), (9, 4, 10, 1.5, 70, 0.6, 200)])
def test_experts_alone(dtype, E, top, F, limit, S, slimit, rows, monkeypatch):
    from types import SimpleNamespace
    from rustinfer_amd.engine import Workspace, make_runtime
    from rustinfer_amd.parts import MoEFeedForward
    rt = make_runtime(dtype, DEV)
    width = 40
    x = some_rows(rows, width, 3)
    part = MoEFeedForward(width, F, E, top, score="sigmoid", weigh_input=True, limit=limit, shared_size=S, shared_gate=S > 0, shared_limit=slimit)
    g = torch.Generator().manual_seed(E + top)
    router = (torch.randn(E, width, generator=g) * 4.0 / math.sqrt(width)).to(torch.bfloat16)      # scores apart: no close calls
    w = load_part(part, E * top, dtype, scale=2.0, replace={"router": router})
    ctx = SimpleNamespace(workspace=Workspace(rt.device))
    out = part.forward(ctx, x.to(DEV, rt.dtype))
    out = (out.double().sum(0) if out.dim() == 3 else out.double()).cpu().numpy()
    mlp, gaps, xs = moe(E, top, F, limit, S, slimit), [], x.double().numpy()
    ref = P.routed_ff(xs, w, mlp, gaps)
    clear = gaps[0] > (1e-5 if dtype == "float32" else 0.05)
    assert clear.mean() > 0.6 and rel(out[clear], ref[clear]) < PART_TOL[dtype]
    # the weights and limits of this test are such that these mistakes would show
    free = P.routed_ff(xs, w, moe(E, top, F, 1e9, S, 1e9))
    assert rel(free, ref) > 2 * PART_TOL["bfloat16"]

    def weighs_outputs(h, w_, mlp_):
        s = P.sigmoid(h @ w_["router"].T)
        y = np.zeros_like(ref)
        for t in range(h.shape[0]):
            for e in np.argsort(-s[t], kind="stable")[:top]:
                y[t] += s[t, e] * P.expert(h[t:t + 1], P._sub(w_, f"e{e}."), limit)[0]
        return y + (P.sigmoid(h @ w_["shared.sg"].T) * P.expert(h, P._sub(w_, "shared."), slimit) if S else 0.0)
    if E > 1:
        assert rel(weighs_outputs(xs, w, mlp), ref) > 2 * PART_TOL["float32"]


@pytest.mark.parametrize("E,top,F,S", [(8, 2, 32, 24), (70, 5, 3, 0), (300, 300, 2, 7), (5, 1, 7, 40)])
def test_the_two_ways_to_route_give_the_same_bits(E, top, F, S):
    from rustinfer_amd.kernels import ops
    g = torch.Generator().manual_seed(E)
    T, width = 37, (E * F + S + 7) // 8 * 8
    both = (torch.randn(T, E + 1, generator=g) * 3.0).to(DEV)
    logits, sg = both[:, :E], both[:, E] if S else None
    gate_up = (torch.randn(T, 2 * E * F + 2 * S, generator=g) * 2.0).to(DEV)
    weights = torch.empty(T, E, device=DEV)
    ops.moe_route(logits, weights, top, score="sigmoid")
    two, one = torch.empty(T, width, device=DEV), torch.empty(T, width, device=DEV)
    clip = ops.ClippedGate(0.9, 1.4)
    ops.moe_swiglu_weighted(gate_up, weights, two, E, F, shared=S, clip=clip, weigh_input=True, shared_gate=sg)
    ops.moe_swiglu_routed(gate_up, logits, one, E, F, top, score="sigmoid", shared=S, clip=clip, weigh_input=True, shared_gate=sg)
    assert torch.equal(one, two)
    s = P.sigmoid(logits.double().cpu().numpy())
    want = np.zeros((T, width))
    gu = gate_up.double().cpu().numpy()
    pair = lambda gt, up, lim: np.minimum(gt, lim) * P.sigmoid(1.702 * np.minimum(gt, lim)) * (np.clip(up, -lim, lim) + 1.0)
    for t in range(T):
        for e in np.argsort(-s[t], kind="stable")[:top]:
            a = gu[t, e * 2 * F:(e + 1) * 2 * F] * s[t, e]
            want[t, e * F:(e + 1) * F] = pair(a[:F], a[F:], 0.9)
        if S:
            a = gu[t, 2 * E * F:]
            want[t, E * F:E * F + S] = pair(a[:S], a[S:], 1.4) * P.sigmoid(sg[t].double().item())
    assert rel(one.double().cpu().numpy(), want) < 2e-6


# ---------------------------------------------------------------------------
# whole models through the engine's step function
# ---------------------------------------------------------------------------
LENGTHS = (70, 3, 121, 1, 38)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["A", "B", "C"])
def test_every_cut_gives_the_plain_logits(tdirs, plain_logits, name, dtype):
    reqs, logits = plain_logits(name, LENGTHS, 21)
    eng = engine_for(tdirs[name], dtype, name)
    for label, steps in (("whole", cut_whole(reqs)), ("last tokens alone", cut_tail_single(reqs, tail=50)),
                         ("portions", cut_portions(reqs, seed=3)),
                         ("portions of two", cut_portions(reqs, seed=4, sizes=(2, 2, 3, 2, 1, 2)))):
        check_rows(steps, run_steps(eng, steps), logits, dtype, f"{name} {dtype} {label}")
        assert not eng.cache.live_requests()


def test_the_stream_after_every_layer(tdirs, plain):
    """The residual stream after each layer against the plain one: names the first layer that differs."""
    from rustinfer_amd.engine import StepEntry
    for name in CONFIGS:
        cfg, w = plain[name]
        toks = random_requests(cfg["vocab"], (45,), 9)["r0"]
        want = []
        P.forward(cfg, w, toks, want)
        eng = engine_for(tdirs[name], "float32", name)
        got = []
        for lay in eng.model.layers:
            def fwd(ctx, hidden, cache, _f=lay.forward, **kw):
                _f(ctx, hidden, cache, **kw)
                x, p = hidden.x.detach().double(), hidden.pending
                if p is not None:
                    x = x + (p.double().sum(0) if p.dim() == 3 else p.double())
                got.append(x.cpu().numpy().copy())
            lay.forward = fwd
        eng.step([StepEntry("r0", toks, list(range(len(toks))))])
        assert len(got) == len(want)
        for i, (a, b) in enumerate(zip(got, want)):
            assert rel(a, b) < 2e-5, (name, i)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["A", "B"])
def test_mixed_batches_with_pages_and_slots_used_again(tdirs, plain_logits, name, dtype):
    from rustinfer_amd.engine import StepEntry
    reqs, logits = plain_logits(name, (90, 17, 64, 5, 130, 33, 2, 71), 22)
    page = PAGE[name]
    max_tokens = 3 * (-(-130 // 64) * 64)
    eng = engine_for(tdirs[name], dtype, name, num_pages=max_tokens // page, max_requests=3, max_len=256)
    steps = cut_mixed(reqs, max_tokens, seed=5, max_live=3, tail=6)
    assert max(len(st["entries"]) for st in steps) == 3
    slots, users, given_back, results = set(), {}, 0, {}
    for st in steps:
        lg = eng.step([StepEntry(e["id"], e["tokens"], e["want"]) for e in st["entries"]])
        slots.update(eng.cache.slot(e["id"]) for e in st["entries"])
        for e in st["entries"]:
            for p in eng.cache.table(0, e["id"]):
                given_back += p < 0
                users.setdefault(p, set()).add(e["id"])
        if lg.shape[0]:
            results[st["step"]] = lg.cpu().numpy()
        for rid in st["end"]:
            eng.release(rid)
    assert len(slots) == 3 and len(reqs) > 3                          # eight requests went through three state slots
    assert any(len(u) > 1 for p, u in users.items() if p >= 0)       # pages were used again
    assert given_back > 0                                             # some of them because a chunk had ended
    check_rows(steps, results, logits, dtype, f"{name} {dtype} mixed")
    eng.cache.check()


@pytest.mark.parametrize("name", ["A", "C"])
def test_a_batch_gives_what_each_request_gives_alone(tdirs, name):
    from rustinfer_amd.engine import StepEntry
    reqs = random_requests(CONFIGS[name]["vocab"], (40, 9, 1, 25), 30)
    eng = engine_for(tdirs[name], "float32", name)
    alone = {}
    for rid, toks in reqs.items():
        if len(toks) > 1:
            eng.step([StepEntry(rid, toks[:-1], [])])
        alone[rid] = eng.step([StepEntry(rid, toks[-1:], [0])]).cpu().numpy()[0]
        eng.release(rid)
    eng.step([StepEntry(rid, toks[:-1], []) for rid, toks in reqs.items() if len(toks) > 1])
    both = eng.step([StepEntry(rid, toks[-1:], [0]) for rid, toks in reqs.items()]).cpu().numpy()
    s = float(np.std(both))
    for row, rid in enumerate(reqs):
        assert np.abs(both[row] - alone[rid]).max() < 1e-4 * s, rid


@pytest.mark.parametrize("name", ["A", "B", "C"])
def test_long_decoding(tdirs, plain, name):
    """Twenty tokens of prompt and 280 single tokens, through every chunk's end, on a pool that holds no more than the
    layer that sees most needs."""
    cfg, w = plain[name]
    toks = random_requests(cfg["vocab"], (300,), 40)["r0"]
    logits = plain_rows(cfg, w, {"r0": toks})
    # the unbounded reader of B keeps every page; A's longest reach is a chunk of 33 (5 pages of 8 and the one begun), C's one of 50
    eng = engine_for(tdirs[name], "float32", name, num_pages={"A": 7, "B": 19, "C": 5}[name])
    steps = cut_tail_single({"r0": toks}, tail=280)
    check_rows(steps, run_steps(eng, steps), logits, "float32", f"{name} long decoding")


@pytest.mark.parametrize("name", ["A", "C"])
def test_greedy_generation_through_the_scheduler(tdirs, plain, name):
    from rustinfer_amd.llm import LLM
    from rustinfer_amd.sampling import SamplingParams
    cfg, w = plain[name]
    prompts = list(random_requests(cfg["vocab"], (12, 47, 5, 30, 21), 50).values())
    llm = LLM(model=tdirs[name], dtype="float32", paged_block_size=PAGE[name], num_blocks=48, max_batch_seqs=3,
              max_model_len=128, max_batch_tokens=64, chunked_prefill_size=32)
    res = llm.generate(prompts, SamplingParams(max_tokens=12, ignore_eos=True))
    for p, r in zip(prompts, res):
        assert len(r.token_ids) == 12
        toks = list(p)
        for i, t in enumerate(r.token_ids):
            row = P.forward(cfg, w, toks)[-1]
            assert row.max() - row[t] < 1e-3 * max(1.0, float(np.std(row))), (i, t, int(np.argmax(row)))
            toks.append(t)
    assert llm.engine.graph_replays > 0 or not llm.engine._graph_sizes


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_decode_steps_replay_a_graph_across_chunk_borders(tdirs, plain, dtype):
    """The captured step of single tokens, replayed while requests of different lengths pass chunk and page borders,
    against eager steps of a second engine."""
    from rustinfer_amd.engine import StepEntry
    cfg, _ = plain["A"]
    reqs = random_requests(cfg["vocab"], (80, 66, 95), 70)
    outs = []
    for graphs in (False, True):
        eng = engine_for(tdirs["A"], dtype, "A")
        eng.enable_graphs(graphs)
        eng.step([StepEntry(rid, toks[:-40], []) for rid, toks in reqs.items()])
        rows = []
        for i in range(40):
            rows.append(eng.step([StepEntry(rid, toks[len(toks) - 40 + i:len(toks) - 39 + i], [0]) for rid, toks in reqs.items()]).cpu().numpy().copy())
        assert (eng.graph_replays > 0) == graphs
        outs.append(np.stack(rows))
    assert np.abs(outs[0] - outs[1]).max() < 1e-5 * np.std(outs[0])


def test_trace_replay_of_a_zotonex_model(tdirs, plain_logits, tmp_path):
    """bin/trace_run as a user starts it, on the mixed cut, four state slots."""
    import subprocess
    import sys
    from helpers import ROOT
    reqs, logits = plain_logits("A", (50, 20, 9, 77, 30), 60)
    steps = cut_mixed(reqs, 512, seed=1, max_live=4, tail=5)
    cmd = [sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model", tdirs["A"], "--dtype", "bfloat16",
           "--out", str(tmp_path), "--max-tokens", "512"]
    proc = subprocess.Popen(cmd, stdin=subprocess.PIPE, stdout=subprocess.PIPE, text=True)
    try:
        for st in steps:
            proc.stdin.write(json.dumps(st) + "\n")
            proc.stdin.flush()
            assert proc.stdout.readline().strip() == f"done {st['step']}"
        proc.stdin.close()
        assert proc.wait(timeout=120) == 0
    finally:
        if proc.poll() is None:
            proc.kill()
    results = {}
    for st in steps:
        n = sum(len(e["want"]) for e in st["entries"])
        if n:
            results[st["step"]] = np.fromfile(os.path.join(str(tmp_path), f"{st['step']}.f32"), dtype="<f4").reshape(n, -1)
    check_rows(steps, results, logits, "bfloat16", "trace replay")


# ---------------------------------------------------------------------------
# configurations drawn at random
# ---------------------------------------------------------------------------
def draw_config(rng):
    """A configuration whose every size, its chunks and its borrowers are drawn."""
    pick = lambda xs: xs[int(rng.integers(0, len(xs)))]
    layers, owners = [], []
    for i in range(int(rng.integers(2, 7))):
        size = lambda: pick([1, 5, 16, 17, 48, 64, 100, 128, 150, 256, None])
        diff = pick([0.0, 0.1, 0.3, 0.55, 0.8])
        if owners and rng.random() < 0.45:
            j = pick(owners)
            o = layers[j]["mixer"]
            mixer = att(o["heads"], o["kv_heads"], o["dim"], o["vdim"], pick([0.1, 0.2]), size(), diff, kv_from=j)
        else:
            H = pick([1, 2, 3, 4, 6, 8, 12])
            mixer = att(H, pick([g for g in (1, 2, 3, 4, 6) if H % g == 0]), pick([8, 16, 20, 32, 48, 64, 96, 128]), pick([16, 24, 32, 64, 96, 128, 160]),
                        pick([0.1, 0.125, 0.2]), size(), diff)
            owners.append(i)
        E = pick([1, 2, 4, 7, 8, 16])
        mlp = None if rng.random() < 0.15 else moe(E, int(rng.integers(1, E + 1)), pick([16, 40, 96, 128]), pick([0.5, 1.0, 2.5, 7.0]),
                                                   pick([0, 24, 96, 256]), pick([0.4, 1.0, 6.0]))
        layers.append(layer(mixer, mlp))
    return dict(architecture="Zotonex", vocab=pick([100, 333, 777, 1000]), width=pick([64, 96, 192, 320, 512]),
                norm=dict(eps=pick([1e-5, 1e-6])), embedding=dict(scale=pick([1.0, 4.0, 12.0])), logit_scale=pick([0.1, 1.0, 3.0]), layers=layers)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("seed", [11, 12, 13, 14, 15, 16, 17, 18])
def test_configurations_drawn_at_random(seed, dtype, tmp_path):
    """Last tokens alone, portions, and a mixed schedule on a pool that is too small for all requests at once, against
    the plain implementation; 32-bit is the sharp test, bfloat16 goes through the kernels that serving uses."""
    from rustinfer_amd.engine import build_engine
    from rustinfer_amd.weights import write_safetensors
    cfg = draw_config(np.random.default_rng(seed))
    with open(tmp_path / "config.json", "w") as f:
        json.dump(cfg, f)
    write_safetensors(str(tmp_path / "model.safetensors"), draw_weights(cfg, seed))
    cfg, w = P.read_model(str(tmp_path))
    reqs = random_requests(cfg["vocab"], (150, 3, 290, 40, 1, 77), seed)
    logits = plain_rows(cfg, w, reqs)
    max_tokens = 2 * 320 + 64
    eng = build_engine(str(tmp_path), dtype=dtype, device=DEV, page_size=16, num_pages=max_tokens // 16, max_requests=4,
                       max_model_len=max_tokens, max_batch_tokens=2048)
    for label, steps in (("last tokens alone", cut_tail_single(reqs, tail=40)), ("portions", cut_portions(reqs, seed=seed)),
                         ("mixed", cut_mixed(reqs, max_tokens, seed=seed, max_live=4, tail=6))):
        check_rows(steps, run_steps(eng, steps), logits, dtype, f"{json.dumps(cfg)} {label}")
        assert not eng.cache.live_requests()
