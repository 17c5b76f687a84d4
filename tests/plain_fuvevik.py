"""A plain, slow implementation of the Fuvevik design in float64 numpy: one function per mechanism, written from
the equations, sharing no code with the engine.  It runs one whole sequence at a time and keeps nothing between
calls; the tests compare the engine's logits, layer outputs and kernels with it.

Notation: ``d`` width, ``T`` tokens of the sequence, weights as stored ([out, in], applied as ``W x``); ``w`` maps
tensor names to arrays, ``pre`` is a layer's prefix (``l3.``).
"""
from __future__ import annotations

import json
import math
import os
import struct
from typing import Dict, List, Optional

import numpy as np

F = np.float64
GLU_SLOPE = 1.702          # the slope inside the experts' sigmoid
SINUSOID_BASE = 10000.0


def rms(x: np.ndarray, eps: float) -> np.ndarray:
    """x / sqrt(mean(x^2) + eps) over the last axis."""
    return x / np.sqrt((x * x).mean(axis=-1, keepdims=True) + eps)


def norm(x: np.ndarray, weight: np.ndarray, eps: float) -> np.ndarray:
    """The layers' norm: its weight is stored as what it differs from one by."""
    return rms(x, eps) * (1.0 + weight)


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


# ------------------------------------------------------------------ embedding

def sinusoid(positions: np.ndarray, d: int) -> np.ndarray:
    """[positions, d]: column 2i is sin(p * base^(-2i / d)), column 2i + 1 the cosine of the same angle."""
    out = np.zeros((len(positions), d), dtype=F)
    for c in range(d):
        angle = positions.astype(F) * SINUSOID_BASE ** (-2.0 * (c // 2) / d)
        out[:, c] = np.cos(angle) if c % 2 else np.sin(angle)
    return out


def embed(tokens: List[int], w: Dict[str, np.ndarray]) -> np.ndarray:
    rows = w["embed"][tokens].astype(F)
    return rows + sinusoid(np.arange(len(tokens)), rows.shape[1])


# ------------------------------------------------------------------ several streams around a sublayer

def sublayer_input(streams: np.ndarray, w: Dict[str, np.ndarray], hc: str) -> np.ndarray:
    """streams [s, T, d] -> [T, d]: their sum with the weights ``hc``.in.  ``hc``: the prefix (``l0.hc1.``)."""
    return np.einsum("s,std->td", w[hc + "in"], streams)


def sublayer_output(streams: np.ndarray, y: np.ndarray, w: Dict[str, np.ndarray], hc: str) -> np.ndarray:
    """New stream t: the sum over the old streams f of mix[f, t] x_f, plus out[t] y."""
    return np.einsum("ft,fnd->tnd", w[hc + "mix"], streams) + w[hc + "out"][:, None, None] * y[None]


# ------------------------------------------------------------------ mixer: attention

def temperature(positions: np.ndarray, q_temp: Optional[dict]) -> np.ndarray:
    """What a query at each position is multiplied by."""
    if q_temp is None:
        return np.ones(len(positions), dtype=F)
    return np.array([1.0 + q_temp["coef"] * math.log((int(p) + 1) // q_temp["every"] + 1) for p in positions], dtype=F)


def sink_softmax(scores: np.ndarray, sink: float) -> np.ndarray:
    """scores [T, T] (query, key): weights over the keys j <= i whose denominator also holds exp(sink), a term without a
    key: a row's weights sum to less than one."""
    T = scores.shape[-1]
    s = np.where(np.tri(T, dtype=bool), scores, -np.inf)
    top = np.maximum(s.max(axis=-1, keepdims=True), sink)
    e = np.exp(s - top)
    return e / (e.sum(axis=-1, keepdims=True) + np.exp(sink - top))


def attention_keys_values(h: np.ndarray, m: dict, w: Dict[str, np.ndarray], pre: str, eps: float):
    """What an attention layer with projections of its own keeps of every token: normed keys [T, G, dim] and values
    [T, G, vdim]."""
    T = h.shape[0]
    G, dk, dv = m["kv_heads"], m["dim"], m["vdim"]
    k = rms((h @ w[pre + "mix.k"].T).reshape(T, G, dk), eps) * w[pre + "mix.k.norm"]
    return k, (h @ w[pre + "mix.v"].T).reshape(T, G, dv)


def attention(h: np.ndarray, kv, m: dict, w: Dict[str, np.ndarray], pre: str, eps: float) -> np.ndarray:
    """``kv``: this layer's own keys and values (``attention_keys_values``), or those of the layer ``kv_from`` names."""
    T = h.shape[0]
    H, G, dk, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    keys, values = kv
    q = rms((h @ w[pre + "mix.q"].T).reshape(T, H, dk), eps) * w[pre + "mix.q.norm"]
    q = q * temperature(np.arange(T), m.get("q_temp"))[:, None, None]
    out = np.zeros((T, H, dv), dtype=F)
    for hd in range(H):
        g = hd // (H // G)
        out[:, hd] = sink_softmax(q[:, hd] @ keys[:, g].T * m["scale"], float(w[pre + "mix.sink"][hd])) @ values[:, g]
    out = out.reshape(T, H * dv) * sigmoid(h @ w[pre + "mix.g"].T)         # one gate a channel
    return out @ w[pre + "mix.o"].T


# ------------------------------------------------------------------ feed-forward

def dense(h: np.ndarray, w: Dict[str, np.ndarray], pre: str) -> np.ndarray:
    return np.maximum(h @ w[pre + "mlp.up"].T, 0.0) ** 2 @ w[pre + "mlp.down"].T


def expert(h: np.ndarray, w: Dict[str, np.ndarray], pre: str, limit: float) -> np.ndarray:
    """``pre``: the expert's prefix (``l0.mlp.e3.``)."""
    g = np.minimum(h @ w[pre + "gate"].T, limit)
    u = np.clip(h @ w[pre + "up"].T, -limit, limit)
    return (g * sigmoid(GLU_SLOPE * g) * (u + 1.0)) @ w[pre + "down"].T


def route(h: np.ndarray, mlp: dict, w: Dict[str, np.ndarray], pre: str, margins: Optional[np.ndarray] = None):
    """(chosen [T, top], weights [T, top]) among the experts and, behind them, the identity experts.  The scores are the
    softmax over all of them; the largest scores plus correction are chosen; the weights are the chosen ones' scores over
    their sum.  ``margins`` [T], if given, is lowered to the gap between the last one chosen and the first one left out,
    taken between the logits' exponentials relative to the larger (a choice made by less than rounding moves the scores
    may fall the other way in an implementation that rounds)."""
    r = mlp["router"]
    E, top = r["experts"] + (r.get("identity") or 0), r["top"]
    z = h @ w[pre + "mlp.router"].T
    assert z.shape[1] == E
    s = np.exp(z - z.max(axis=1, keepdims=True))
    s = s / s.sum(axis=1, keepdims=True)
    choice = s + w[pre + "mlp.correction"]
    order = np.argsort(-choice, axis=1, kind="stable")
    chosen = order[:, :top]
    if margins is not None and top < E:
        last = np.take_along_axis(choice, order[:, top - 1:top], axis=1)[:, 0]
        first_out = np.take_along_axis(choice, order[:, top:top + 1], axis=1)[:, 0]
        size = np.maximum(np.take_along_axis(s, order[:, top - 1:top], axis=1)[:, 0], np.take_along_axis(s, order[:, top:top + 1], axis=1)[:, 0])
        np.minimum(margins, (last - first_out) / size, out=margins)
    weights = np.take_along_axis(s, chosen, axis=1)
    return chosen, weights / (weights.sum(axis=1, keepdims=True) + 1e-20)


def routed(h: np.ndarray, mlp: dict, w: Dict[str, np.ndarray], pre: str, margins: Optional[np.ndarray] = None) -> np.ndarray:
    chosen, weights = route(h, mlp, w, pre, margins)
    out = np.zeros_like(h)
    for t in range(h.shape[0]):
        for e, a in zip(chosen[t], weights[t]):
            if e < mlp["router"]["experts"]:
                out[t] += a * expert(h[t:t + 1], w, f"{pre}mlp.e{e}.", mlp["expert"]["limit"])[0]
            else:
                out[t] += a * h[t]                                          # an identity expert: the input itself
    if mlp.get("shared") is not None:
        out = out + expert(h, w, pre + "mlp.shared.", mlp["shared"]["limit"])
    return out


def feed_forward(h: np.ndarray, mlp: dict, w: Dict[str, np.ndarray], pre: str, margins: Optional[np.ndarray] = None) -> np.ndarray:
    return dense(h, w, pre) if mlp["kind"] == "dense" else routed(h, mlp, w, pre, margins)


# ------------------------------------------------------------------ the model

def forward(cfg: dict, w: Dict[str, np.ndarray], tokens: List[int], layers_out: Optional[list] = None,
            margins: Optional[np.ndarray] = None) -> np.ndarray:
    """Logits [T, vocab] of one whole sequence.  ``layers_out``, if a list, gets the sum of the streams behind every layer;
    ``margins`` [T] (start it at infinity) the smallest gap by which any router chose for each token (see ``route``)."""
    eps = cfg["norm"]["eps"]
    w = {k: np.asarray(v, dtype=F) for k, v in w.items()}
    streams = np.repeat(embed(tokens, w)[None], cfg["streams"], axis=0)
    kept: Dict[int, tuple] = {}
    for i, layer in enumerate(cfg["layers"]):
        pre, m = f"l{i}.", layer["mixer"]
        if layer["type"] != "attention":
            raise ValueError(f"layer type {layer['type']!r}")
        h = norm(sublayer_input(streams, w, pre + "hc1."), w[pre + "norm1"], eps)
        if m.get("kv_from") is None:
            kept[i] = attention_keys_values(h, m, w, pre, eps)
        y = attention(h, kept[i if m.get("kv_from") is None else m["kv_from"]], m, w, pre, eps)
        streams = sublayer_output(streams, y, w, pre + "hc1.")
        if layer.get("mlp") is not None:
            h = norm(sublayer_input(streams, w, pre + "hc2."), w[pre + "norm2"], eps)
            streams = sublayer_output(streams, feed_forward(h, layer["mlp"], w, pre, margins), w, pre + "hc2.")
        if layers_out is not None:
            layers_out.append(streams.sum(axis=0))
    return norm(streams.sum(axis=0), w["final.norm"], eps) @ w["embed"].T


# ------------------------------------------------------------------ reading a model folder

def read_safetensors(path: str) -> Dict[str, np.ndarray]:
    out = {}
    with open(path, "rb") as fh:
        (n,) = struct.unpack("<Q", fh.read(8))
        header = json.loads(fh.read(n))
        data = fh.read()
    for name, meta in header.items():
        if name == "__metadata__":
            continue
        a, b = meta["data_offsets"]
        raw = data[a:b]
        if meta["dtype"] == "BF16":
            arr = (np.frombuffer(raw, dtype="<u2").astype(np.uint32) << 16).view(np.float32)
        elif meta["dtype"] == "F32":
            arr = np.frombuffer(raw, dtype="<f4")
        elif meta["dtype"] == "I32":
            arr = np.frombuffer(raw, dtype="<i4")
        else:
            raise ValueError(f"{name}: stored type {meta['dtype']}")
        out[name] = arr.reshape(meta["shape"]).astype(F)
    return out


def read_model_folder(folder: str):
    with open(os.path.join(folder, "config.json")) as fh:
        cfg = json.load(fh)
    return cfg, read_safetensors(os.path.join(folder, "model.safetensors"))
