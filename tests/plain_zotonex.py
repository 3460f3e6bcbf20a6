"""A plain, slow implementation of the Zotonex decoder: whole sequences, no cache, no batches,
64-bit arithmetic, one function for each mechanism, and no code shared with ``rustinfer_amd``.

The design in this file's own notation.  ``x`` is the residual stream,
``unit(y) = y / sqrt(mean(y^2) + eps)``.

* embedding: ``x = E[token] * embedding.scale``;
* a layer: ``x <- x + mixer(unit(x) * n1)``, then, if it has a feed-forward,
  ``x <- x + ff(unit(x) * n2)``;
* mixer ``attention`` makes every head's output from the difference of two softmax maps over one
  set of values: a query head holds two queries and a key head two keys (first map, second map),
  each ``dim`` wide, brought to unit size and multiplied by a weight that all heads and both maps
  share; no rotation.  Positions are cut into chunks of ``mask.size`` counted from the sequence's
  start, and a query sees the keys of its own chunk up to itself.  With the maps' outputs ``a``,
  ``b`` and one number a layer ``lam = exp(lq1 . lk1) - exp(lq2 . lk2) + diff``, a head's output is
  ``unit(a - lam b) * (1 - diff)``.  A layer with ``kv_from: j`` reads layer j's keys and values;
* feed-forward ``moe``: an expert's gate row is clipped from above at ``limit``, its up row to
  ``[-limit, limit]``, and ``g sigmoid(1.702 g) (u + 1)`` goes through the down matrix; the ``top``
  experts with the largest ``sigmoid`` of the router's logits run on the token's row multiplied by
  that score; a shared expert's output, times the sigmoid of one more logit, is added;
* output: ``logits = W_head (unit(x) * n) * logit_scale``.
"""
from __future__ import annotations

import json
import os
import struct
from typing import Dict, List, Optional

import numpy as np

GATE_SLOPE = 1.702


# ---------------------------------------------------------------------------
# reading a model folder (a reader of its own)
# ---------------------------------------------------------------------------
def read_safetensors(path: str) -> Dict[str, np.ndarray]:
    with open(path, "rb") as f:
        (hlen,) = struct.unpack("<Q", f.read(8))
        header = json.loads(f.read(hlen))
        data = f.read()
    out = {}
    for name, info in header.items():
        if name == "__metadata__":
            continue
        b, e = info["data_offsets"]
        raw, dt = data[b:e], info["dtype"]
        if dt == "F32":
            arr = np.frombuffer(raw, dtype="<f4").astype(np.float64)
        elif dt == "BF16":
            arr = (np.frombuffer(raw, dtype="<u2").astype(np.uint32) << 16).view(np.float32).astype(np.float64)
        elif dt == "I32":
            arr = np.frombuffer(raw, dtype="<i4").astype(np.int64)
        else:
            raise ValueError(f"{name}: dtype {dt}")
        out[name] = arr.reshape(info["shape"])
    return out


def read_model(model_dir: str):
    with open(os.path.join(model_dir, "config.json")) as f:
        cfg = json.load(f)
    return cfg, read_safetensors(os.path.join(model_dir, "model.safetensors"))


# ---------------------------------------------------------------------------
# small functions
# ---------------------------------------------------------------------------
def unit(y: np.ndarray, eps: float) -> np.ndarray:
    return y / np.sqrt(np.mean(y * y, axis=-1, keepdims=True) + eps)


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def softmax_rows(s: np.ndarray) -> np.ndarray:
    e = np.exp(s - np.max(s, axis=-1, keepdims=True))
    return e / np.sum(e, axis=-1, keepdims=True)


def chunk_mask(T: int, size: Optional[int]) -> np.ndarray:
    """[T, T]: may row i see column j?"""
    i, j = np.arange(T)[:, None], np.arange(T)[None, :]
    seen = j <= i
    return seen if not size else seen & (i // size == j // size)


# ---------------------------------------------------------------------------
# the mixer
# ---------------------------------------------------------------------------
def one_map(q, k, v, scale, seen):
    """One softmax map of one head: q [T, dim], k [T, dim], v [T, vdim]."""
    return softmax_rows(np.where(seen, (q @ k.T) * scale, -np.inf)) @ v


def keys_values(h, w, m, eps):
    """What a layer keeps for itself and for layers that borrow from it: keys [T, G, 2, dim] and
    values [T, G, vdim]."""
    T, G = h.shape[0], m["kv_heads"]
    k = unit((h @ w["k"].T).reshape(T, G, 2, m["dim"]), eps) * w["k.norm"]
    return k, (h @ w["v"].T).reshape(T, G, m["vdim"])


def map_weight(w, diff: float) -> float:
    """How much of the second map is taken off the first."""
    return float(np.exp(np.sum(w["lq1"] * w["lk1"])) - np.exp(np.sum(w["lq2"] * w["lk2"])) + diff)


def difference(a, b, lam: float, diff: float, eps: float):
    return unit(a - lam * b, eps) * (1.0 - diff)


def attention(h, w, m, eps, kv):
    T, H, G = h.shape[0], m["heads"], m["kv_heads"]
    k, v = kv
    q = unit((h @ w["q"].T).reshape(T, H, 2, m["dim"]), eps) * w["q.norm"]
    mask = m.get("mask")
    seen = chunk_mask(T, mask["size"] if mask else None)
    lam, heads = map_weight(w, m["diff"]), []
    for i in range(H):
        g = i // (H // G)
        a, b = (one_map(q[:, i, s], k[:, g, s], v[:, g], m["scale"], seen) for s in (0, 1))
        heads.append(difference(a, b, lam, m["diff"], eps))
    return np.concatenate(heads, axis=1) @ w["o"].T


# ---------------------------------------------------------------------------
# the feed-forward
# ---------------------------------------------------------------------------
def expert(h, w, limit: float):
    g = np.minimum(h @ w["gate"].T, limit)
    u = np.clip(h @ w["up"].T, -limit, limit)
    return (g * sigmoid(GATE_SLOPE * g) * (u + 1.0)) @ w["down"].T


def routed_ff(h, w, mlp, gaps=None):
    """``gaps`` (a list) receives, for every row, how far the last chosen expert's logit lies above the
    first one left out (infinite where all experts are chosen)."""
    E, top = mlp["router"]["experts"], mlp["router"]["top"]
    z = h @ w["router"].T
    s = sigmoid(z)
    if gaps is not None:
        ranked = -np.sort(-z, axis=1)
        gaps.append(ranked[:, top - 1] - ranked[:, top] if top < E else np.full(h.shape[0], np.inf))
    out = np.zeros((h.shape[0], w["e0.down"].shape[0]))
    for t in range(h.shape[0]):
        for e in np.argsort(-s[t], kind="stable")[:top]:
            out[t] += expert(s[t, e] * h[t:t + 1], _sub(w, f"e{e}."), mlp["expert"]["limit"])[0]
    if mlp.get("shared"):
        out += sigmoid(h @ w["shared.sg"].T) * expert(h, _sub(w, "shared."), mlp["shared"]["limit"])
    return out


# ---------------------------------------------------------------------------
# the model
# ---------------------------------------------------------------------------
def _sub(w: Dict[str, np.ndarray], prefix: str) -> Dict[str, np.ndarray]:
    return {k[len(prefix):]: a for k, a in w.items() if k.startswith(prefix)}


def forward(cfg: dict, w: Dict[str, np.ndarray], ids, layers_out: Optional[List[np.ndarray]] = None,
            gaps: Optional[List[np.ndarray]] = None) -> np.ndarray:
    """Logits [T, vocab] of one sequence from its first token.  ``layers_out`` collects the
    residual stream after every layer, ``gaps`` every routed layer's margins (``routed_ff``)."""
    eps = cfg["norm"]["eps"]
    x = w["embed"][np.asarray(ids, dtype=np.int64)] * cfg["embedding"]["scale"]
    kept = {}
    for i, layer in enumerate(cfg["layers"]):
        mw, m = _sub(w, f"l{i}.mix."), layer["mixer"]
        if layer["type"] != "attention":
            raise ValueError(layer["type"])
        h = unit(x, eps) * w[f"l{i}.norm1"]
        source = m.get("kv_from")
        if source is None:
            kept[i] = keys_values(h, mw, m, eps)
        x = x + attention(h, mw, m, eps, kept[i if source is None else source])
        if layer.get("mlp") is not None:
            x = x + routed_ff(unit(x, eps) * w[f"l{i}.norm2"], _sub(w, f"l{i}.mlp."), layer["mlp"], gaps)
        if layers_out is not None:
            layers_out.append(x.copy())
    return (unit(x, eps) * w["final.norm"]) @ w["head"].T * cfg["logit_scale"]


def greedy(logits: np.ndarray) -> int:
    return int(np.argmax(logits))
