"""A plain, slow implementation of the Sibodra decoder: whole sequences, no cache, no batches,
64-bit arithmetic, one function for each mechanism, and no code shared with ``rustinfer_amd``.

The design in this file's own notation.  ``unit(y) = y / sqrt(mean(y^2) + eps)``, ``center(y) = y - mean(y)``.

* hyper-connections: the residual stream is ``n`` rows ``X_1 .. X_n`` a token, all ``E[token]`` at first.  A sub-layer ``f``
  (the mixer, then the feed-forward if there is one) with a vector ``a [n]``, a vector ``b [n]`` and a matrix
  ``M [n, n]`` reads ``f(norm(sum_s a_s X_s))`` and leaves ``X'_t = sum_s M_st X_s + b_t f(..)``; the model's
  output is made from ``sum_t X_t``;
* norm: ``unit(center(x)) * w``, no bias;
* mixer ``attention``: grouped softmax attention over all earlier positions; queries and keys are unit-normed per head,
  multiplied by a weight of the head's size and turned over their first ``rot.dims`` features (feature i with
  i + dims/2, llama3-scaled frequencies); scores pass ``c tanh(s / c)``; the softmax's denominator has 1 added; each
  head's output is multiplied by one sigmoid a head;
* mixer ``latent_attention``: queries from a normed latent of their own, keys and values from another normed latent,
  beside one turned key part for all heads; the heads' outputs are multiplied by sigmoids feature by feature;
* feed-forward ``dense``: ``W_down (silu(W_gate h) * W_up h)``; ``moe``: experts ``W_down relu(W_up h)^2`` of which the ``top``
  with the largest logits ``W_router h + b`` are summed with the softmax over those logits, and a shared expert;
* output: ``c tanh(W_head norm(.) / c)``.
"""
from __future__ import annotations

import json
import math
import os
import struct
from typing import Dict, List, Optional

import numpy as np


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


def layer_norm(x: np.ndarray, w: np.ndarray, eps: float) -> np.ndarray:
    c = x - np.mean(x, axis=-1, keepdims=True)
    return c / np.sqrt(np.mean(c * c, axis=-1, keepdims=True) + eps) * w


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def silu(z):
    return z * sigmoid(z)


def softcap(z, cap: Optional[float]):
    return z if not cap else cap * np.tanh(z / cap)


def frequencies(rot: dict) -> np.ndarray:
    """base^(-2i/dims), stretched band by band if the rotation has ``scaling``."""
    dims, f = rot["dims"], []
    sc = rot.get("scaling")
    for i in range(dims // 2):
        fi = rot["base"] ** (-2.0 * i / dims)
        if sc:
            wavelength = 2.0 * math.pi / fi
            if wavelength > sc["original"] / sc["low"]:
                fi = fi / sc["factor"]
            elif wavelength >= sc["original"] / sc["high"]:
                s = (sc["original"] / wavelength - sc["low"]) / (sc["high"] - sc["low"])
                fi = (1.0 - s) * fi / sc["factor"] + s * fi
        f.append(fi)
    return np.array(f)


def rotate(y: np.ndarray, rot: Optional[dict]) -> np.ndarray:
    """y [T, n]: the first ``dims`` features turned by the row's position, feature i with i + dims/2."""
    if not rot:
        return y
    h = rot["dims"] // 2
    ang = np.arange(y.shape[0])[:, None] * frequencies(rot)[None, :]
    c, s = np.cos(ang), np.sin(ang)
    u, v = y[:, :h], y[:, h:2 * h]
    return np.concatenate([u * c - v * s, v * c + u * s, y[:, 2 * h:]], axis=1)


def causal_mask(T: int) -> np.ndarray:
    return np.tril(np.ones((T, T), dtype=bool))


def softmax_attention(q, k, v, scale, cap=None, one_more=False):
    """q [T, dk], k [T, dk], v [T, dv] of one head: row i sees rows j <= i.  ``one_more``: the denominator
    has 1 added (a key of score 0 without a value)."""
    s = softcap((q @ k.T) * scale, cap)
    s = np.where(causal_mask(q.shape[0]), s, -np.inf)
    top = np.max(s, axis=1, keepdims=True)
    if one_more:
        top = np.maximum(top, 0.0)
    e = np.exp(s - top)
    den = np.sum(e, axis=1, keepdims=True)
    if one_more:
        den = den + np.exp(-top)
    return (e / den) @ v


# ---------------------------------------------------------------------------
# mixers
# ---------------------------------------------------------------------------
def head_gated_attention(h, w, m, eps):
    T, H, G, d, dv = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = unit((h @ w["q"].T).reshape(T, H, d), eps) * w["q.norm"]
    k = unit((h @ w["k"].T).reshape(T, G, d), eps) * w["k.norm"]
    v = (h @ w["v"].T).reshape(T, G, dv)
    gate = sigmoid(h @ w["g"].T)
    rot, outs = m.get("rot"), []
    for i in range(H):
        g = i // (H // G)
        o = softmax_attention(rotate(q[:, i], rot), rotate(k[:, g], rot), v[:, g], m["scale"], m.get("softcap"), one_more=True)
        outs.append(o * gate[:, i:i + 1])
    return np.concatenate(outs, axis=1) @ w["o"].T


def latent_attention(h, w, m, eps):
    T, H, d, r, dv, R = h.shape[0], m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    cq = unit(h @ w["dq"].T, eps) * w["dq.norm"]
    q = (cq @ w["uq"].T).reshape(T, H, d + r)
    down = h @ w["dkv"].T
    c = unit(down[:, :R], eps) * w["dkv.norm"]
    k_rot = rotate(down[:, R:], m["rot"])
    k_up = (c @ w["uk"].T).reshape(T, H, d)
    v = (c @ w["uv"].T).reshape(T, H, dv)
    outs = []
    for i in range(H):
        qi = np.concatenate([q[:, i, :d], rotate(q[:, i, d:], m["rot"])], axis=1)
        ki = np.concatenate([k_up[:, i], k_rot], axis=1)
        outs.append(softmax_attention(qi, ki, v[:, i], m["scale"]))
    return (np.concatenate(outs, axis=1) * sigmoid(h @ w["g"].T)) @ w["o"].T


MIXERS = {"attention": head_gated_attention, "latent_attention": latent_attention}


# ---------------------------------------------------------------------------
# feed-forwards
# ---------------------------------------------------------------------------
def gated_ff(h, w):
    return (silu(h @ w["gate"].T) * (h @ w["up"].T)) @ w["down"].T


def expert(h, w):
    return (np.maximum(h @ w["up"].T, 0.0) ** 2) @ w["down"].T


def chosen_weights(z: np.ndarray, top: int):
    """(indices of the ``top`` largest logits, their softmax among themselves)."""
    idx = np.argsort(-z, kind="stable")[:top]
    e = np.exp(z[idx] - np.max(z[idx]))
    return idx, e / np.sum(e)


def routed_ff(h, w, mlp, gaps=None):
    """``gaps`` (a list) receives, for every row, how far the last chosen expert's logit lies above the first
    one left out (infinite where all experts are chosen)."""
    E, top = mlp["router"]["experts"], mlp["router"]["top"]
    z = h @ w["router"].T + w["router.b"]
    if gaps is not None:
        ranked = -np.sort(-z, axis=1)
        gaps.append(ranked[:, top - 1] - ranked[:, top] if top < E else np.full(h.shape[0], np.inf))
    out = expert(h, _sub(w, "shared.")) if mlp.get("shared") else np.zeros((h.shape[0], w["e0.down"].shape[0]))
    for t in range(h.shape[0]):
        for e, p in zip(*chosen_weights(z[t], top)):
            out[t] += p * expert(h[t:t + 1], _sub(w, f"e{e}."))[0]
    return out


# ---------------------------------------------------------------------------
# hyper-connections and the model
# ---------------------------------------------------------------------------
def read_streams(X: np.ndarray, a: np.ndarray) -> np.ndarray:
    """X [T, n, width] -> the row a sub-layer (its norm) reads."""
    return np.sum(a[None, :, None] * X, axis=1)


def write_streams(X: np.ndarray, M: np.ndarray, b: np.ndarray, y: np.ndarray) -> np.ndarray:
    """All streams at once from the old ones: M is indexed [from, to]."""
    out = np.zeros_like(X)
    for t in range(X.shape[1]):
        for s in range(X.shape[1]):
            out[:, t] += M[s, t] * X[:, s]
        out[:, t] += b[t] * y
    return out


def _sub(w: Dict[str, np.ndarray], prefix: str) -> Dict[str, np.ndarray]:
    return {k[len(prefix):]: a for k, a in w.items() if k.startswith(prefix)}


def forward(cfg: dict, w: Dict[str, np.ndarray], ids, layers_out: Optional[List[np.ndarray]] = None,
            gaps: Optional[List[np.ndarray]] = None) -> np.ndarray:
    """Logits [T, vocab] of one sequence from its first token.  ``layers_out`` collects the sum of the streams
    after every layer, ``gaps`` every routed layer's margins (``routed_ff``)."""
    eps, n = cfg["norm"]["eps"], cfg["streams"]
    x = w["embed"][np.asarray(ids, dtype=np.int64)]
    X = np.repeat(x[:, None, :], n, axis=1)
    for i, layer in enumerate(cfg["layers"]):
        hc, mlp = _sub(w, f"l{i}.hc1."), layer.get("mlp")
        h = layer_norm(read_streams(X, hc["in"]), w[f"l{i}.norm1"], eps)
        X = write_streams(X, hc["mix"], hc["out"], MIXERS[layer["type"]](h, _sub(w, f"l{i}.mix."), layer["mixer"], eps))
        if mlp is not None:
            hc, fw = _sub(w, f"l{i}.hc2."), _sub(w, f"l{i}.mlp.")
            h = layer_norm(read_streams(X, hc["in"]), w[f"l{i}.norm2"], eps)
            X = write_streams(X, hc["mix"], hc["out"], gated_ff(h, fw) if mlp["kind"] == "dense" else routed_ff(h, fw, mlp, gaps))
        if layers_out is not None:
            layers_out.append(np.sum(X, axis=1))
    z = layer_norm(np.sum(X, axis=1), w["final.norm"], eps) @ w["head"].T
    return softcap(z, cfg.get("logit_softcap"))


def greedy(logits: np.ndarray) -> int:
    return int(np.argmax(logits))
