"""Sibodra on the GPU against the plain implementation (``plain_sibodra.py``): every mechanism alone, then whole models of
three small configurations that differ in every size, in the number of residual rows and in the order of their layers,
through every way of cutting requests into steps, through pages and slots that are used again, and through
``LLM.generate``.  Weights are drawn here with deviations that make activations of order one; some tests build inputs so
that one far key decides, and plant mistakes in the plain implementation to see that they could tell."""
import json
import math
import os
from types import SimpleNamespace

import numpy as np
import pytest
import torch

import plain_sibodra as P
from helpers import cut_mixed, cut_portions, cut_tail_single, cut_whole, random_requests, run_steps
from test_gpu_belorax import CUTS, PART_TOL, Rows, check_rows, portion_kernel, rel, run_part, some_rows  # noqa: F401

pytestmark = pytest.mark.gpu
DEV = "cuda:0"
SCALING = dict(factor=4.0, low=1.0, high=8.0, original=90)


def att(heads, kv, dim, vdim, scale, cap=9.0, dims=None, base=300.0, scaling=None):
    m = dict(heads=heads, kv_heads=kv, dim=dim, vdim=vdim, scale=scale, rot=dict(base=base, dims=dims or dim))
    if cap:
        m["softcap"] = cap
    if scaling:
        m["rot"]["scaling"] = scaling
    return m


def lat(heads, dim, rot_dim, vdim, q_rank, kv_rank, scale, base=200.0, dims=None):
    return dict(heads=heads, dim=dim, rot_dim=rot_dim, vdim=vdim, q_rank=q_rank, kv_rank=kv_rank, scale=scale,
                rot=dict(base=base, dims=dims or rot_dim))


def dense(ff):
    return dict(kind="dense", ff=ff)


def moe(experts, top, ff, shared_ff):
    d = dict(kind="moe", expert=dict(ff=ff), router=dict(experts=experts, top=top))
    if shared_ff:
        d["shared"] = dict(ff=shared_ff)
    return d


def layer(mixer, mlp):
    return dict(type="latent_attention" if "kv_rank" in mixer else "attention", mixer=mixer, mlp=mlp)


CONFIGS = {
    # three residual rows, a layer without feed-forward, rotations over a part of the head and over all of it
    "A": dict(architecture="Sibodra", vocab=200, width=72, streams=3, norm=dict(eps=1e-5), logit_softcap=6.0, layers=[
        layer(lat(4, 12, 8, 20, 40, 28, 0.25), moe(5, 2, 24, 40)),
        layer(att(4, 2, 12, 20, 0.4, 5.0, 8, 100.0, SCALING), dense(88)),
        layer(att(2, 1, 24, 16, 0.3, 3.0), None),
        layer(lat(3, 8, 16, 12, 24, 20, 0.3, dims=12), moe(4, 1, 16, 8)),
    ]),
    # heads beyond one 64-wide slice, more experts than a wave has lanes, no shared expert, one residual row
    "B": dict(architecture="Sibodra", vocab=333, width=136, streams=1, norm=dict(eps=1e-6), logit_softcap=20.0, layers=[
        layer(att(8, 2, 40, 132, 0.2, 30.0, 24), moe(70, 3, 16, 56)),
        layer(att(3, 3, 72, 40, 0.15, 8.0, 72, 5000.0, SCALING), moe(9, 4, 32, 0)),
        layer(lat(8, 32, 16, 72, 64, 136, 0.12), moe(6, 6, 48, 24)),
        layer(lat(1, 40, 64, 130, 96, 72, 0.1), dense(120)),
    ]),
    # a width and a vocabulary that are no multiples of eight, odd head sizes, more heads than a call of the kernels takes
    "C": dict(architecture="Sibodra", vocab=211, width=100, streams=5, norm=dict(eps=1e-6), logit_softcap=4.0, layers=[
        layer(att(3, 1, 6, 10, 0.7, 2.0, 2), dense(60)),
        layer(lat(40, 6, 2, 3, 18, 14, 0.4), moe(8, 3, 10, 6)),
        layer(att(5, 5, 18, 14, 0.4, None, 10), moe(3, 2, 30, 12)),
        layer(lat(5, 10, 6, 14, 7, 9, 0.35, dims=4), None),
        layer(att(16, 1, 8, 12, 0.5, 4.0, 6, 40.0, SCALING), moe(7, 1, 9, 33)),
    ]),
}
PAGE = {"A": 8, "B": 16, "C": 16}


def bf16_round(a: np.ndarray) -> torch.Tensor:
    return torch.tensor(a, dtype=torch.float32).to(torch.bfloat16)


def draw_weights(cfg: dict, seed: int):
    """name -> bfloat16 tensor for every tensor of the design: activations of order one, scores that reach the cap, gates
    and mixing weights that all differ."""
    rng = np.random.default_rng(seed)
    W, n = cfg["width"], cfg["streams"]
    mat = lambda o, i, s=1.0: bf16_round(s * rng.standard_normal((o, i)) / math.sqrt(i))
    vec = lambda k, mean, std: bf16_round(mean + std * rng.standard_normal(k))
    t = {"embed": bf16_round(rng.standard_normal((cfg["vocab"], W))), "final.norm": vec(W, 1.0, 0.2), "head": mat(cfg["vocab"], W, 2.0)}
    for i, lay in enumerate(cfg["layers"]):
        m, p, mlp = lay["mixer"], f"l{i}.", lay["mlp"]
        for q in (1, 2) if mlp is not None else (1,):
            t[p + f"norm{q}"] = vec(W, 1.0, 0.2)
            t[p + f"hc{q}.in"], t[p + f"hc{q}.out"] = vec(n, 1.0 / n, 0.4), vec(n, 0.7, 0.3)
            t[p + f"hc{q}.mix"] = bf16_round(0.7 * np.eye(n) + 0.4 / math.sqrt(n) * rng.standard_normal((n, n)))
        H, dv = m["heads"], m["vdim"]
        if lay["type"] == "attention":
            t[p + "mix.q"], t[p + "mix.q.norm"] = mat(H * m["dim"], W), vec(m["dim"], 1.5, 0.3)
            t[p + "mix.k"], t[p + "mix.k.norm"] = mat(m["kv_heads"] * m["dim"], W), vec(m["dim"], 1.5, 0.3)
            t[p + "mix.v"], t[p + "mix.g"] = mat(m["kv_heads"] * dv, W), mat(H, W, 2.0)
        else:
            t[p + "mix.dq"], t[p + "mix.dq.norm"] = mat(m["q_rank"], W), vec(m["q_rank"], 1.0, 0.3)
            t[p + "mix.uq"] = mat(H * (m["dim"] + m["rot_dim"]), m["q_rank"], 1.5)
            t[p + "mix.dkv"], t[p + "mix.dkv.norm"] = mat(m["kv_rank"] + m["rot_dim"], W), vec(m["kv_rank"], 1.0, 0.3)
            t[p + "mix.uk"], t[p + "mix.uv"] = mat(H * m["dim"], m["kv_rank"], 1.5), mat(H * dv, m["kv_rank"])
            t[p + "mix.g"] = mat(H * dv, W, 2.0)
        t[p + "mix.o"] = mat(W, H * dv, 1.5)
        if mlp is None:
            continue
        if mlp["kind"] == "dense":
            t[p + "mlp.gate"], t[p + "mlp.up"], t[p + "mlp.down"] = mat(mlp["ff"], W), mat(mlp["ff"], W), mat(W, mlp["ff"], 2.0)
            continue
        E, F = mlp["router"]["experts"], mlp["expert"]["ff"]
        t[p + "mlp.router"], t[p + "mlp.router.b"] = mat(E, W, 2.0), vec(E, 0.5, 1.0)
        for name, size in [(f"e{e}", F) for e in range(E)] + ([("shared", mlp["shared"]["ff"])] if mlp.get("shared") else []):
            t[p + f"mlp.{name}.up"], t[p + f"mlp.{name}.down"] = mat(size, W), mat(W, size)
    return t


@pytest.fixture(scope="module")
def tdirs(tmp_path_factory):
    from rustinfer_amd.weights import write_safetensors
    out = {}
    for k, (name, cfg) in enumerate(CONFIGS.items()):
        d = str(tmp_path_factory.mktemp("sibodra_" + name))
        with open(os.path.join(d, "config.json"), "w") as f:
            json.dump(cfg, f)
        write_safetensors(os.path.join(d, "model.safetensors"), draw_weights(cfg, 71 + k))
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
        rows.margin[rid] = np.min(np.stack(gaps), axis=0) / 4.0 if gaps else np.full(len(toks), np.inf)
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
def rotary_of(m, size):
    from rustinfer_amd.config import RopeScaling
    from rustinfer_amd.parts import RotaryEmbedding
    sc = m["rot"].get("scaling")
    scaling = RopeScaling("llama3", sc["factor"], sc["low"], sc["high"], sc["original"]) if sc else None
    return RotaryEmbedding(size, m["rot"]["base"], scaling=scaling, rot_dim=m["rot"]["dims"])


def attention_part(width, m, eps=1e-5):
    from rustinfer_amd.parts import WindowAttention
    pe = rotary_of(m, m["dim"])
    return WindowAttention(width, m["heads"], m["kv_heads"], m["dim"], m["vdim"], m["scale"], qk_norm_eps=eps, pos_enc=pe,
                           sink_score=0.0, softcap=m.get("softcap"), head_gate=True), [pe]


def latent_part(width, m, eps=1e-5):
    from rustinfer_amd.parts import LatentAttention
    pe = rotary_of(m, m["rot_dim"])
    return LatentAttention(width, m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"], m["scale"], eps, pos_enc=pe,
                           interleaved=False, q_rank=m["q_rank"], output_gate=True), [pe]


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
            wt[n] = (torch.randn(s.shape, generator=g) * 0.8).to(torch.bfloat16)
    for n, t in dict(replace).items():
        assert n in wt and tuple(wt[n].shape) == tuple(t.shape)
        wt[n] = t.to(torch.bfloat16)
    part.load(wt, make_runtime(dtype, DEV))
    return {n: t.double().numpy() for n, t in wt.items()}


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("H,G,dk,dv,scale,cap,dims,scaling", [
    (4, 2, 16, 24, 0.4, 3.0, 8, SCALING), (3, 3, 40, 36, 0.2, 50.0, 40, None), (8, 1, 32, 16, 0.3, 2.0, 2, None), (2, 2, 128, 128, 0.09, 5.0, 64, SCALING),
    (5, 5, 72, 200, 0.12, None, 30, None), (6, 1, 24, 40, 0.3, 1.0, 24, SCALING), (2, 1, 256, 256, 0.06, 8.0, 128, None), (1, 1, 6, 2, 0.8, 4.0, 4, None),
    (32, 1, 8, 12, 0.5, 6.0, 8, None), (6, 2, 64, 128, 0.12, 20.0, 16, SCALING), (20, 1, 24, 72, 0.25, 3.0, 6, None), (3, 1, 10, 100, 0.5, 2.5, 10, None),
    (6, 3, 48, 40, 0.2, 4.0, 32, SCALING), (2, 1, 200, 24, 0.1, 6.0, 176, None), (5, 1, 8, 16, 0.5, 3.0, 4, None)])
def test_capped_attention_alone(dtype, H, G, dk, dv, scale, cap, dims, scaling, portion_kernel):
    d, m = 48, att(H, G, dk, dv, scale, cap, dims, 50.0, scaling)
    part, pes = attention_part(d, m)
    w = load_part(part, H * dk + dv, dtype, scale=2.0)
    x = some_rows(sum(CUTS), d, 5)
    ref = P.head_gated_attention(x.double().numpy(), w, m, 1e-5)
    page = 16 if portion_kernel == "parts" else 8
    assert rel(run_part(part, pes, dtype, x, CUTS, page=page), ref) < PART_TOL[dtype]
    other = some_rows(60, d, 8)
    assert rel(run_part(part, pes, dtype, x, CUTS, page=page, batch_with=other), ref) < PART_TOL[dtype]     # another request beside it


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("H,d,r,dv,Q,R,dims", [
    (3, 8, 4, 12, 30, 20, 4), (8, 32, 16, 24, 80, 72, 16), (1, 12, 6, 10, 5, 9, 2), (5, 40, 16, 72, 33, 136, 12), (16, 16, 8, 24, 64, 48, 8),
    (2, 64, 64, 130, 200, 192, 64), (32, 4, 2, 4, 12, 6, 2), (40, 8, 4, 6, 24, 12, 4), (4, 24, 32, 40, 48, 64, 32)])
def test_latent_attention_alone(dtype, H, d, r, dv, Q, R, dims, portion_kernel):
    width, m = 56, lat(H, d, r, dv, Q, R, 0.4 / math.sqrt(d + r), 60.0, dims)
    part, pes = latent_part(width, m)
    w = load_part(part, H * d + R, dtype, scale=2.0)
    x = some_rows(sum(CUTS), width, 6)
    ref = P.latent_attention(x.double().numpy(), w, m, 1e-5)
    assert rel(run_part(part, pes, dtype, x, CUTS, page=16 if portion_kernel == "parts" else 8), ref) < PART_TOL[dtype]
    assert rel(run_part(part, pes, dtype, x, [sum(CUTS)], page=16, batch_with=some_rows(3, width, 9)), ref) < PART_TOL[dtype]


@pytest.mark.parametrize("mistake", ["no cap", "no sink", "gate of another head", "norm weights left out", "every feature turned", "scaling left out"])
def test_the_attention_test_could_tell(mistake, monkeypatch):
    """Mistakes planted in the plain implementation move its result far beyond the tolerances above."""
    d, m = 48, att(4, 2, 16, 24, 0.4, 3.0, 8, 50.0, SCALING)
    part, _ = attention_part(d, m)
    g = torch.Generator().manual_seed(1)
    w = {n: torch.randn(s.shape, generator=g).double().numpy() * (2.0 / math.sqrt(d) if len(s.shape) == 2 else 0.3) for n, s in part.param_specs().items()}
    w["q.norm"], w["k.norm"] = 1.0 + w["q.norm"], 1.0 + w["k.norm"]
    x = some_rows(80, d, 5).double().numpy()
    ref = P.head_gated_attention(x, w, m, 1e-5)
    keep = P.softmax_attention
    if mistake == "no cap":
        m = dict(m, softcap=None)
    elif mistake == "no sink":
        monkeypatch.setattr(P, "softmax_attention", lambda *a, one_more=False, **k: keep(*a, **k))
    elif mistake == "gate of another head":
        w = dict(w, g=np.roll(w["g"], 1, axis=0))
    elif mistake == "norm weights left out":
        w = dict(w, **{"k.norm": np.ones(16)})
    elif mistake == "every feature turned":
        m = dict(m, rot=dict(m["rot"], dims=16))
    else:
        m = dict(m, rot=dict(m["rot"], scaling=None))
    assert rel(P.head_gated_attention(x, w, m, 1e-5), ref) > 2 * PART_TOL["bfloat16"]


def test_the_latent_test_could_tell(monkeypatch):
    width, m = 56, lat(3, 8, 4, 12, 30, 20, 0.12, 60.0, 4)
    part, _ = latent_part(width, m)
    g = torch.Generator().manual_seed(2)
    w = {n: torch.randn(s.shape, generator=g).double().numpy() * (2.0 / math.sqrt(s.shape[1]) if len(s.shape) == 2 else 0.3) for n, s in part.param_specs().items()}
    w["dq.norm"], w["dkv.norm"] = 1.0 + w["dq.norm"], 1.0 + w["dkv.norm"]
    x = some_rows(80, width, 5).double().numpy()
    ref = P.latent_attention(x, w, m, 1e-5)
    for wrong in (dict(w, **{"dq.norm": np.ones(30)}), dict(w, **{"dkv.norm": np.ones(20)}), dict(w, g=np.roll(w["g"], 12, axis=0)), dict(w, uq=np.roll(w["uq"], 12, axis=0))):
        assert rel(P.latent_attention(x, wrong, m, 1e-5), ref) > 2 * PART_TOL["bfloat16"]
    monkeypatch.setattr(P, "rotate", lambda y, rot: y)
    assert rel(P.latent_attention(x, w, m, 1e-5), ref) > 2 * PART_TOL["bfloat16"]


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_the_added_one_decides_where_scores_are_low(dtype, portion_kernel):
    """Keys that point away from every query: scores near minus the cap, so that a sequence's first tokens return
    almost nothing and later ones a share that grows with the number of keys."""
    d, H = 16, 2
    m = att(H, 1, d, 8, 1.0, 4.0, 2, 1e6)
    part, pes = attention_part(d, m)
    eye = torch.eye(d)
    w = load_part(part, 4, dtype, replace={"q": torch.cat([eye, eye]), "k": -eye, "q.norm": torch.ones(d), "k.norm": torch.ones(d)})
    x = (torch.ones(sum(CUTS), d) + 0.2 * some_rows(sum(CUTS), d, 3)).to(torch.bfloat16).float()
    ref = P.head_gated_attention(x.double().numpy(), w, m, 1e-5)
    without = P.softmax_attention(np.ones((3, 2)), -np.ones((3, 2)), np.ones((3, 1)), 4.0, 4.0)
    assert np.allclose(without, 1.0) and np.abs(ref[0]).max() < 0.05 * np.abs(ref[-1]).max()
    got = run_part(part, pes, dtype, x, CUTS, page=16 if portion_kernel == "parts" else 8)
    assert rel(got, ref) < PART_TOL[dtype]
    assert np.abs(got[:4] - ref[:4]).max() < 4 * PART_TOL[dtype] * np.abs(ref[:4]).max()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("decoded", [False, True])
@pytest.mark.parametrize("kind", ["attention", "latent"])
def test_one_key_decides(dtype, decoded, kind, portion_kernel):
    """Queries that match one key each, far back, at pages' borders, the first positions of the sequence, the query's own
    position and the one before: a key that is lost, or read at another place, changes these rows beyond any rounding."""
    T, dk = 420, 24
    pairs = {2: 0, 3: 3, 40: 1, 317: 15, 318: 16, 333: 0, 350: 31, 351: 32, 380: 379, 390: 390, 399: 128, 411: 300}
    keys = sorted(set(pairs.values()))
    feat = {k: n for n, k in enumerate(keys)}
    assert len(feat) == 11
    look, eye = torch.zeros(dk, dk), torch.eye(dk)
    x = 0.05 * torch.randn(T, dk, generator=torch.Generator().manual_seed(2))
    x[:, 11:22] = 0.0
    x[:, 22] = 1.0
    for k, n in feat.items():
        look[n, 11 + n] = 1.0                              # a query reads feature 11 + n into key feature n
        x[k, :11] = 0.0
        x[k, n] = 4.0
    for q, k in pairs.items():
        x[q, 11 + feat[k]] += 4.0
    x = x.to(torch.bfloat16).float()
    if kind == "attention":
        m = att(1, 1, dk, 12, 2.0, 60.0, 2, 1e8)
        shift = torch.zeros(dk, dk)                        # the turned features stay out of it
        shift[2:, :22] = torch.eye(22)
        part, pes = attention_part(dk, m, eps=1e-6)
        w = load_part(part, 5, dtype, replace={"q": shift @ look, "k": shift @ eye, "q.norm": torch.ones(dk), "k.norm": torch.ones(dk)})
        plainly = P.head_gated_attention
    else:
        m = lat(1, dk, 2, 12, dk, dk, 2.0, 1e8)
        part, pes = latent_part(dk, m, eps=1e-6)
        down = torch.cat([eye, torch.zeros(2, dk)])
        w = load_part(part, 5, dtype, replace={"dq": eye, "uq": torch.cat([look, torch.zeros(2, dk)]), "dkv": down, "uk": eye,
                                               "dq.norm": torch.ones(dk), "dkv.norm": torch.ones(dk)})
        plainly = P.latent_attention
    xs = x.double().numpy()
    ref = plainly(xs, w, m, 1e-6)
    size = np.abs(ref).max()
    for q, k in pairs.items():                             # the test can tell: without that key's row the output is another
        if k != q:
            off = xs.copy()
            off[k] = xs[(k + 7) % T if (k + 7) % T not in feat else (k + 8) % T]
            assert np.abs(plainly(off[:q + 1], w, m, 1e-6)[q] - ref[q]).max() > 0.1 * size, (q, k)
    cuts = [310] + [1] * 110 if decoded else [310, 17, 2, 40, 11, 2, 38]
    got = run_part(part, pes, dtype, x, cuts, page=16)
    for q in pairs:
        assert np.abs(got[q] - ref[q]).max() < PART_TOL[dtype] * size, q


def test_thousands_of_keys():
    """A prompt of 4,300 tokens and single tokens behind it, more stretches of keys than a row may leave partial results
    of; every query has a favourite far back, and positions run far past the stretched rotation's bands."""
    T, d = 4330, 32
    m = att(4, 2, 16, 24, 1.2, 12.0, 12, 10000.0, SCALING)
    part, pes = attention_part(d, m)
    w = load_part(part, 3, "bfloat16", scale=2.0)
    x = some_rows(T, d, 11)
    ref = P.head_gated_attention(x.double().numpy(), w, m, 1e-5)
    got = run_part(part, pes, "bfloat16", x, [2048, 2200, 52] + [1] * 30, page=16, num_pages=300, max_len=4400)
    assert rel(got[:4100], ref[:4100]) < PART_TOL["bfloat16"] and rel(got[4100:], ref[4100:]) < PART_TOL["bfloat16"]


def test_capped_scores_and_weights_keep_their_32_bits(monkeypatch):
    """The bfloat16 matrix-instruction kernels against the 32-bit ones on the same bfloat16 queries, keys, values and gates:
    far closer than scores or weights rounded to bfloat16 would be, in portions and in single tokens."""
    from rustinfer_amd.kernels import ops
    d, m = 48, att(4, 2, 64, 64, 0.3, 6.0, 32)
    x = some_rows(sum(CUTS), d, 5)
    outs = []
    real = ops.window_attention
    for parts in (True, False):
        monkeypatch.setattr(ops, "WINDOW_ATTENTION_PARTS", parts)
        keep = []

        def both(q, out, *args, **kw):
            real(q, out, *args, **kw)
            keep.append(out.double().cpu().numpy().copy())
        monkeypatch.setattr(ops, "window_attention", both)
        part, pes = attention_part(d, m)
        load_part(part, 5, "bfloat16", scale=2.0)
        run_part(part, pes, "bfloat16", x, CUTS, page=16)
        outs.append(np.concatenate(keep))
    diff = np.abs(outs[0] - outs[1])
    # results that round to neighbouring bfloat16 numbers now and then, almost never further apart
    assert (diff > 0).mean() < 0.02 and diff.max() < 2.0 ** -7 * np.abs(outs[1]).max()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("T", [1, 5, 16, 17, 70, 131])
@pytest.mark.parametrize("H,N,K,tail,rot", [(3, 20, 8, 6, 4), (2, 64, 32, 16, 16), (5, 70, 13, 3, 2), (1, 33, 40, 5, 0), (4, 128, 64, 0, 0),
                                            (3, 33, 24, 8, 4), (2, 100, 40, 8, 8), (3, 7, 8, 0, 0)])
def test_head_product_with_tail_and_gate(dtype, T, H, N, K, tail, rot):
    from rustinfer_amd.kernels import ops
    dt = getattr(torch, dtype)
    g = torch.Generator().manual_seed(T + N)
    draw = lambda *s: torch.randn(s, generator=g).to(torch.bfloat16).float()
    x, w, gate = draw(T, H * (K + tail)), draw(H, N, K), draw(T, H * N)
    pos = torch.randint(0, 500, (T,), generator=g, dtype=torch.int32)
    ang = torch.arange(500.0)[:, None] * torch.tensor([1.0 / (i + 1) for i in range(max(rot // 2, 1))])[None]
    cos, sin = ang.cos(), ang.sin()
    out = torch.zeros(T, H * (N + tail), device=DEV, dtype=dt)
    rotary = (cos.to(DEV), sin.to(DEV), rot) if rot else None
    ops.head_linear(x.to(DEV, dt), K + tail, w.to(DEV, dt), out, N + tail, tail=tail, rotary=rotary, positions=pos.to(DEV), gate=gate.to(DEV, dt))
    xs = x.double().view(T, H, K + tail)
    y = torch.einsum("thk,hnk->thn", xs[:, :, :K], w.double()) * torch.sigmoid(gate.double()).view(T, H, N)
    t = xs[:, :, K:].clone()
    if rot:
        h, c, s = rot // 2, cos.double()[pos.long()][:, None], sin.double()[pos.long()][:, None]
        a, b = xs[:, :, K:K + h], xs[:, :, K + h:K + rot]
        t[:, :, :h], t[:, :, h:rot] = a * c - b * s, b * c + a * s
    want = torch.cat([y, t], dim=2).reshape(T, -1).numpy()
    assert rel(out.double().cpu().numpy(), want) < {"float32": 2e-6, "bfloat16": 5e-3}[dtype]


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("E,top,F,S,rows", [(4, 1, 24, 40, 70), (16, 3, 56, 8, 5), (70, 3, 16, 33, 100), (6, 6, 8, 24, 33), (3, 2, 41, 0, 1),
                                            (130, 8, 4, 12, 17), (1, 1, 32, 16, 65), (9, 4, 10, 70, 200)])
def test_experts_alone(dtype, E, top, F, S, rows):
    from rustinfer_amd.engine import Workspace, make_runtime
    from rustinfer_amd.parts import MoEFeedForward
    rt = make_runtime(dtype, DEV)
    width = 40
    x = some_rows(rows, width, 3)
    part = MoEFeedForward(width, F, E, top, score="chosen_softmax", router_bias=True, gated=False, shared_size=S)
    g = torch.Generator().manual_seed(E + top)
    router = (torch.randn(E, width, generator=g) * 4.0 / math.sqrt(width)).to(torch.bfloat16)      # logits apart: few close calls
    w = load_part(part, E * top, dtype, scale=2.0, replace={"router": router})
    ctx = SimpleNamespace(workspace=Workspace(rt.device))
    out = part.forward(ctx, x.to(DEV, rt.dtype))
    out = (out.double().sum(0) if out.dim() == 3 else out.double()).cpu().numpy()
    mlp, gaps, xs = moe(E, top, F, S), [], x.double().numpy()
    ref = P.routed_ff(xs, w, mlp, gaps)
    clear = gaps[0] > (1e-5 if dtype == "float32" else 0.05)
    assert clear.mean() > 0.6 and rel(out[clear], ref[clear]) < PART_TOL[dtype]
    if top < E and rows > 3:                             # the bias decides with these weights
        assert rel(P.routed_ff(xs, dict(w, **{"router.b": np.zeros(E)}), mlp), ref) > 2 * PART_TOL["bfloat16"]


@pytest.mark.parametrize("E,top,F,S", [(8, 2, 32, 24), (70, 5, 3, 0), (300, 300, 2, 7), (5, 1, 7, 40)])
def test_the_two_ways_to_route_give_the_same_bits(E, top, F, S):
    from rustinfer_amd.kernels import ops
    g = torch.Generator().manual_seed(E)
    T, width = 37, (E * F + S + 7) // 8 * 8
    logits = (torch.randn(T, E, generator=g) * 30.0).to(DEV)
    logits[3] -= 500.0                                   # far below zero: softmax values that would all underflow
    bias = torch.randn(E, generator=g).to(DEV)
    up = (torch.randn(T, E * F + S, generator=g) * 2.0).to(DEV)
    weights = torch.empty(T, E, device=DEV)
    ops.moe_route(logits, weights, top, score="chosen_softmax", bias=bias)
    two, one = torch.empty(T, width, device=DEV), torch.empty(T, width, device=DEV)
    ops.moe_swiglu_weighted(up, weights, two, E, F, shared=S, gated=False)
    ops.moe_swiglu_routed(up, logits, one, E, F, top, score="chosen_softmax", shared=S, gated=False, bias=bias)
    assert torch.equal(one, two)
    z = (logits.double() + bias.double()).cpu().numpy()
    u = np.maximum(up.double().cpu().numpy(), 0.0) ** 2
    want = np.zeros((T, width))
    for t in range(T):
        for e, p in zip(*P.chosen_weights(z[t], top)):
            want[t, e * F:(e + 1) * F] = p * u[t, e * F:(e + 1) * F]
        want[t, E * F:E * F + S] = u[t, E * F:]
    assert rel(one.double().cpu().numpy(), want) < 1e-5        # (32-bit logits of up to 500 carry 3e-5)


@pytest.mark.parametrize("n", [1, 2, 3, 4, 5, 8])
@pytest.mark.parametrize("d,T,parts,act", [(72, 9, 1, "float32"), (101, 300, 3, "bfloat16"), (1536, 5, 8, "bfloat16"), (4100, 260, 2, "float32"), (5000, 3, 6, "float32"),
                                           (256, 700, 1, "bfloat16")])
def test_streams_kernel(n, d, T, parts, act):
    """Reading, mixing and norming the residual rows: in place, from rows that are all one, a selection of rows, partial
    sums, with and without a norm's bias, as layer norm and as RMS norm."""
    from rustinfer_amd.kernels import ops
    g = torch.Generator().manual_seed(n * d)
    r = lambda *s: torch.randn(s, generator=g)
    X, delta = r(T, n, d) + 0.5, r(parts, T, d)
    mix, out_w, in_w, w, b = r(n, n), r(n), r(n), 1.0 + 0.2 * r(d), 0.3 * r(d)
    f64 = lambda t: t.double().numpy()
    y = f64(delta).sum(0)
    tol = {"float32": 3e-6, "bfloat16": 5e-3}[act]
    dev = lambda t: t.to(DEV).contiguous()
    how = dict(mix=dev(mix), out_w=dev(out_w))
    buf = lambda k: torch.full((k, d), 7.0, device=DEV, dtype=getattr(torch, act))
    nump = lambda t: t.double().cpu().numpy()
    dl = dev(delta) if parts > 1 else dev(delta[0])

    def plain(old, bias=True, centered=True):
        new = P.write_streams(old, f64(mix), f64(out_w), y)
        u = P.read_streams(new, f64(in_w))
        act_ = (P.layer_norm(u, f64(w), 1e-5) if centered else P.unit(u, 1e-5) * f64(w)) + (f64(b) if bias else 0.0)
        return new, act_
    new, want = plain(f64(X))
    x, a = dev(X), buf(T)
    ops.hyper_streams(x, n, dev(in_w), dev(w), 1e-5, a, delta=dl, bias=dev(b), streams_out=x, **how)         # in place
    assert rel(nump(x), new) < 3e-6 and rel(nump(a), want) < tol
    x, a = dev(X), buf(T)
    ops.hyper_streams(x, n, dev(in_w), dev(w), 1e-5, a, delta=dl, centered=False, **how)                     # nothing kept
    assert torch.equal(x.cpu(), X) and rel(nump(a), plain(f64(X), bias=False, centered=False)[1]) < tol
    one, a, kept = dev(X[:, 0]), buf(T), torch.empty(T, n, d, device=DEV)
    new1, want1 = plain(np.repeat(f64(X[:, :1]), n, axis=1))
    ops.hyper_streams(one, n, dev(in_w), dev(w), 1e-5, a, delta=dl, bias=dev(b), streams_out=kept, **how)    # all rows are one row
    assert rel(nump(kept), new1) < 3e-6 and rel(nump(a), want1) < tol
    rows = torch.randperm(T, generator=g)[:max(1, T // 2)].to(torch.int32)
    a, kept = buf(rows.numel()), torch.empty(rows.numel(), n, d, device=DEV)
    ops.hyper_streams(dev(X), n, dev(in_w), dev(w), 1e-5, a, delta=dl, bias=dev(b), streams_out=kept, rows=rows.to(DEV), **how)
    assert rel(nump(kept), new[rows.numpy()]) < 3e-6 and rel(nump(a), want[rows.numpy()]) < tol
    a = buf(T)
    ops.hyper_streams(dev(X), n, dev(in_w), dev(w), 1e-5, a)                                                 # no sub-layer has run yet
    assert rel(nump(a), P.layer_norm(P.read_streams(f64(X), f64(in_w)), f64(w), 1e-5)) < tol


def test_streams_kernel_refuses_what_does_not_fit():
    from rustinfer_amd.kernels import ops
    x, a, v = torch.zeros(4, 2, 16, device=DEV), torch.zeros(4, 16, device=DEV), torch.zeros(2, device=DEV)
    w = torch.ones(16, device=DEV)
    for bad in (dict(n=3), dict(in_w=torch.zeros(3, device=DEV)), dict(act=torch.zeros(3, 16, device=DEV)), dict(delta=torch.zeros(4, 16, device=DEV)),
                dict(streams_out=x, rows=torch.arange(4, device=DEV, dtype=torch.int32))):
        kw = dict(x=x, n=2, in_w=v, weight=w, eps=1e-5, act=a)
        kw.update(bad)
        with pytest.raises(ops.KernelError):
            ops.hyper_streams(**kw)
    with pytest.raises(ops.KernelError):
        ops.hyper_streams(torch.zeros(4, 9, 16, device=DEV), 9, torch.zeros(9, device=DEV), w, 1e-5, a)


def test_layer_norm_without_a_bias():
    from rustinfer_amd.kernels import ops
    x, w = some_rows(33, 200, 1) + 3.0, 1.0 + 0.1 * some_rows(1, 200, 2)[0]
    out = torch.empty(33, 200, device=DEV)
    ops.layer_norm(x.to(DEV), w.to(DEV), None, 1e-5, out)
    assert rel(out.double().cpu().numpy(), P.layer_norm(x.double().numpy(), w.double().numpy(), 1e-5)) < 2e-6


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


def total_of(hidden):
    """The sum of the residual rows behind a layer, the last sub-layer's result joined."""
    p = hidden.pending
    d = p.delta.double().sum(0) if p.delta.dim() == 3 else p.delta.double()
    c = p.connection
    X = p.streams.double() if p.streams is not None else hidden.x.double()[:, None].expand(-1, c.streams, -1)
    return (torch.matmul(c.mix.double().t().contiguous(), X) + c.out_w.double()[None, :, None] * d[:, None]).sum(1).cpu().numpy()


def test_the_stream_after_every_layer(tdirs, plain):
    """The sum of the residual rows after each layer against the plain one: names the first layer that differs."""
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
                got.append(total_of(hidden))
            lay.forward = fwd
        eng.step([StepEntry("r0", toks, list(range(len(toks))))])
        assert len(got) == len(want)
        for i, (a, b) in enumerate(zip(got, want)):
            assert rel(a, b) < 2e-5, (name, i)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["A", "C"])
def test_a_few_wanted_rows_of_a_prompt(tdirs, plain_logits, name, dtype):
    """Prompts of which few places are wanted, out of order, or none: the last feed-forward then runs on those rows alone."""
    from rustinfer_amd.engine import StepEntry
    reqs, logits = plain_logits(name, LENGTHS, 21)
    eng = engine_for(tdirs[name], dtype, name)
    steps = []
    for rid, toks in reqs.items():
        if len(toks) < 10:
            continue
        a, b = toks[:len(toks) // 2], toks[len(toks) // 2:]
        steps += [{"step": len(steps), "entries": [{"id": rid, "tokens": a, "want": []}], "end": []},
                  {"step": len(steps) + 1, "entries": [{"id": rid, "tokens": b, "want": [len(b) - 1, 2, 5]}], "end": [rid]}]
    check_rows(steps, run_steps(eng, steps), logits, dtype, f"{name} {dtype} few wanted")


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
    users, results = {}, {}
    for st in steps:
        lg = eng.step([StepEntry(e["id"], e["tokens"], e["want"]) for e in st["entries"]])
        for e in st["entries"]:
            for g in eng.cache.groups:
                for p in eng.cache.table(g.index, e["id"]):
                    users.setdefault((g.index, p), set()).add(e["id"])
        if lg.shape[0]:
            results[st["step"]] = lg.cpu().numpy()
        for rid in st["end"]:
            eng.release(rid)
    assert any(len(u) > 1 for u in users.values())                   # pages were used again
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
    """Twenty tokens of prompt and 280 single tokens on a pool that holds just them."""
    cfg, w = plain[name]
    toks = random_requests(cfg["vocab"], (300,), 40)["r0"]
    logits = plain_rows(cfg, w, {"r0": toks})
    eng = engine_for(tdirs[name], "float32", name, num_pages=-(-300 // PAGE[name]))
    steps = cut_tail_single({"r0": toks}, tail=280)
    check_rows(steps, run_steps(eng, steps), logits, "float32", f"{name} long decoding")


@pytest.mark.parametrize("name", ["A", "B"])
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
@pytest.mark.parametrize("name", ["A", "B"])
def test_decode_steps_replay_a_graph(tdirs, name, dtype):
    """The captured step of single tokens, replayed while requests of different lengths pass page borders, against eager
    steps of a second engine."""
    from rustinfer_amd.engine import StepEntry
    reqs = random_requests(CONFIGS[name]["vocab"], (80, 66, 95), 70)
    outs = []
    for graphs in (False, True):
        eng = engine_for(tdirs[name], dtype, name)
        eng.enable_graphs(graphs)
        eng.step([StepEntry(rid, toks[:-40], []) for rid, toks in reqs.items()])
        rows = []
        for i in range(40):
            rows.append(eng.step([StepEntry(rid, toks[len(toks) - 40 + i:len(toks) - 39 + i], [0]) for rid, toks in reqs.items()]).cpu().numpy().copy())
        assert (eng.graph_replays > 0) == graphs
        outs.append(np.stack(rows))
    assert np.abs(outs[0] - outs[1]).max() < 1e-5 * np.std(outs[0])


def test_trace_replay_of_a_sibodra_model(tdirs, plain_logits, tmp_path):
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
    """A configuration whose every size and constant is drawn."""
    pick = lambda xs: xs[int(rng.integers(0, len(xs)))]
    layers = []
    for i in range(int(rng.integers(2, 6))):
        scaling = pick([None, dict(factor=pick([2.0, 8.0]), low=1.0, high=pick([2.0, 4.0]), original=pick([64, 256, 700]))])
        if rng.random() < 0.5:
            H, dk = pick([1, 2, 3, 4, 6, 8, 12]), pick([8, 16, 20, 32, 48, 64, 96, 128])
            mixer = att(H, pick([g for g in (1, 2, 3, 4, 6) if H % g == 0]), dk, pick([16, 24, 32, 64, 96, 128, 160]), pick([0.1, 0.125, 0.2]),
                        pick([2.0, 8.0, 30.0]), pick([dk, dk // 2, dk // 4 * 2]), pick([100.0, 10000.0, 500000.0]), scaling)
        else:
            r = pick([8, 16, 32, 64])
            mixer = lat(pick([1, 2, 3, 4, 6, 8, 12]), pick([16, 32, 64, 24]), r, pick([16, 40, 64, 96]), pick([24, 64, 160, 200]), pick([32, 72, 128, 192]),
                        pick([0.1, 0.15]), pick([100.0, 10000.0]))
        E = pick([1, 2, 4, 7, 8, 16])
        mlp = None if rng.random() < 0.15 else dense(pick([64, 100, 256])) if rng.random() < 0.3 else moe(E, int(rng.integers(1, E + 1)), pick([16, 40, 96, 128]), pick([0, 24, 96, 256]))
        layers.append(layer(mixer, mlp))
    return dict(architecture="Sibodra", vocab=pick([100, 333, 777, 1000]), width=pick([64, 96, 192, 328, 512]), streams=pick([1, 2, 3, 4, 6]),
                norm=dict(eps=pick([1e-5, 1e-6])), logit_softcap=pick([3.0, 10.0, 30.0]), layers=layers)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("seed", [21, 22, 23, 24, 25, 26, 27, 28])
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
