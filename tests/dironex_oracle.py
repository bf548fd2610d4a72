"""Dironex in plain float64 NumPy: every mechanism as one function over a whole sequence, without caches, batches or kernels.  It shares nothing with the
product path (uzu_amd/, csrc/): the tests hold the engine to these equations.

Notation: T positions, d = model width, h [T, d] what a sublayer reads.  Weights are dicts of float64 arrays keyed by the tensor names of a model directory
(linear weights [out, in]); `cfg` is the parsed config.json.
"""
from __future__ import annotations

import json
import math
import os
from typing import Dict, List, Optional, Tuple

import numpy as np


def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def softplus(z):
    return np.logaddexp(0.0, z)


def rms_norm(x, w, eps: float):
    """x / sqrt(mean(x^2) + eps) * w over the last axis"""
    return x / np.sqrt((x ** 2).mean(axis=-1, keepdims=True) + eps) * w


def causal_conv(h, w):
    """h [T, C], w [C, taps]: out_t = sum_j w[:, j] * h_(t - taps + 1 + j), zeros in front of the sequence (the last tap weighs the current position)"""
    T, taps = h.shape[0], w.shape[1]
    padded = np.concatenate([np.zeros((taps - 1, h.shape[1])), h])
    return sum(padded[j:j + T] * w[:, j] for j in range(taps))


# ------------------------------------------------------------------------------------------------ hyper-connections: `s` copies of the stream
def hyper_read(xs, w_in):
    """xs [s, T, d] -> the row a sublayer reads, sum_s w_in[s] x_s"""
    return np.tensordot(w_in, xs, axes=(0, 0))


def hyper_write(xs, w_mix, w_out, y, mult: float):
    """x_t <- sum_s w_mix[s, t] x_s + mult * w_out[t] * y, every new stream from the old ones"""
    new = np.empty_like(xs)
    for t in range(xs.shape[0]):
        new[t] = mult * w_out[t] * y
        for s in range(xs.shape[0]):
            new[t] += w_mix[s, t] * xs[s]
    return new


# ------------------------------------------------------------------------------------------------ rotation
def rotation_frequencies(dims: int, base: float, scaling: Optional[dict]) -> Tuple[np.ndarray, float]:
    """(angle per position of pair i, factor on cos and sin); `scaling`: YaRN's ramp between the plain and the stretched frequency"""
    f = np.array([base ** (-2.0 * i / dims) for i in range(dims // 2)])
    if not scaling:
        return f, 1.0
    factor, original = float(scaling["factor"]), float(scaling["original"])
    turn = lambda t: dims * math.log(original / (2.0 * math.pi * t)) / (2.0 * math.log(base))
    lo = max(math.floor(turn(float(scaling["fast"]))), 0)
    hi = min(math.ceil(turn(float(scaling["slow"]))), dims - 1)
    ramp = np.clip((np.arange(dims // 2) - lo) / max(hi - lo, 0.001), 0.0, 1.0)
    return f / factor * ramp + f * (1.0 - ramp), 0.1 * math.log(factor) + 1.0


def rotate_half(x, positions, rot: dict):
    """x [..., T, dims]: coordinates (i, i + dims / 2) turn by position * frequency_i"""
    dims = int(rot["dims"])
    f, m = rotation_frequencies(dims, float(rot["base"]), rot.get("scaling"))
    a = np.asarray(positions, dtype=np.float64)[:, None] * f
    c, s = np.cos(a) * m, np.sin(a) * m
    u, v = x[..., :dims // 2], x[..., dims // 2:dims]
    return np.concatenate([u * c - v * s, v * c + u * s, x[..., dims:]], axis=-1)


# ------------------------------------------------------------------------------------------------ mixers
def softmax_attention(scores, visible, values):
    """scores [T, T] (row = query), visible [T, T] bool, values [T, n]"""
    z = np.where(visible, scores, -np.inf)
    z = z - z.max(axis=-1, keepdims=True)
    p = np.exp(z)
    return (p / p.sum(axis=-1, keepdims=True)) @ values


def causal_window(T: int, size: Optional[int] = None):
    """row i sees j <= i, and with a size only the last `size` positions (itself included)"""
    back = np.arange(T)[:, None] - np.arange(T)[None, :]
    return (back >= 0) & (back < size) if size else back >= 0


def latent_attention(h, w: Dict[str, np.ndarray], p: str, mx: dict, eps: float):
    H, dim, rd, vd, rank = (int(mx[k]) for k in ("heads", "dim", "rot_dim", "vdim", "kv_rank"))
    T = h.shape[0]
    pos = np.arange(T)
    cq = rms_norm(h @ w[p + "dq"].T, w[p + "dq.norm"], eps)
    q = (cq @ w[p + "uq"].T).reshape(T, H, dim + rd)
    ckv = h @ w[p + "dkv"].T
    c = rms_norm(ckv[:, :rank], w[p + "dkv.norm"], eps)
    kr = rotate_half(ckv[:, rank:], pos, mx["rot"])
    k = (c @ w[p + "uk"].T).reshape(T, H, dim)
    v = (c @ w[p + "uv"].T).reshape(T, H, vd)
    out = np.empty((T, H, vd))
    for a in range(H):
        qr = rotate_half(q[:, a, dim:], pos, mx["rot"])
        scores = (q[:, a, :dim] @ k[:, a].T + qr @ kr.T) * float(mx["scale"])
        out[:, a] = softmax_attention(scores, causal_window(T), v[:, a])
    out = out.reshape(T, H * vd) * sigmoid(h @ w[p + "g"].T)
    return out @ w[p + "o"].T


def grouped_attention(h, w, p: str, mx: dict, eps: float):
    H, G, dim, vd = (int(mx[k]) for k in ("heads", "kv_heads", "dim", "vdim"))
    T = h.shape[0]
    q = rms_norm((h @ w[p + "q"].T).reshape(T, H, dim), w[p + "q.norm"], eps)
    k = rms_norm((h @ w[p + "k"].T).reshape(T, G, dim), w[p + "k.norm"], eps)
    v = (h @ w[p + "v"].T).reshape(T, G, vd)
    size = (mx.get("mask") or {}).get("size")
    out = np.empty((T, H, vd))
    for a in range(H):
        g = a // (H // G)
        out[:, a] = softmax_attention(q[:, a] @ k[:, g].T * float(mx["scale"]), causal_window(T, size), v[:, g])
    return out.reshape(T, H * vd) @ w[p + "o"].T


# ------------------------------------------------------------------------------------------------ feed-forward
def xielu(z, pq):
    pos, neg = softplus(pq[0]), 0.5 + softplus(pq[1])
    m = np.minimum(z, 0.0)
    return np.where(z > 0, pos * z * z, neg * (np.expm1(m) - m)) + 0.5 * z


def dense_mlp(h, w, p: str):
    return xielu(h @ w[p + "up"].T, w[p + "act"]) @ w[p + "down"].T


def route(h, w, p: str, router: dict):
    """-> chosen experts [T, top] and their weights [T, top]"""
    E, top, scale = int(router["experts"]), int(router["top"]), float(router["scale"])
    groups = router.get("groups") or {"count": 1, "keep": 1}
    count, keep = int(groups["count"]), int(groups["keep"])
    s = sigmoid(h @ w[p + "router"].T)
    ids, weights = [], []
    for row in s:
        choice = row + w[p + "correction"]
        parts = choice.reshape(count, E // count)
        strength = np.sort(parts, axis=1)[:, ::-1][:, :2].sum(axis=1)
        kept = np.argsort(-strength, kind="stable")[:keep]
        masked = np.full_like(parts, -np.inf)
        masked[kept] = parts[kept]
        best = np.argsort(-masked.reshape(E), kind="stable")[:top]
        ids.append(best)
        weights.append(row[best] / (row[best].sum() + 1e-20) * scale)
    return np.array(ids), np.array(weights)


def experts_mlp(h, w, p: str, ml: dict):
    ids, weights = route(h, w, p, ml["router"])
    y = np.zeros_like(h)
    for t in range(h.shape[0]):
        for e, wt in zip(ids[t], weights[t]):
            y[t] += wt * (w[f"{p}e{e}.down"] @ np.maximum(w[f"{p}e{e}.up"] @ h[t], 0.0) ** 2)
    return y


# ------------------------------------------------------------------------------------------------ the model
def layer_order(cfg: dict) -> List[int]:
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return list(range(n))
    a, b, times = int(loop["start"]), int(loop["stop"]), int(loop["times"])
    return list(range(a)) + list(range(a, b)) * times + list(range(b, n))


def forward(cfg: dict, w: Dict[str, np.ndarray], tokens) -> Tuple[np.ndarray, List[np.ndarray]]:
    """-> logits [T, vocab], the sum of the streams behind every layer run"""
    eps, mult = float(cfg["norm"]["eps"]), float(cfg["residual_mult"])
    x0 = w["embed"][np.asarray(tokens, dtype=np.int64)] * float(cfg["embedding"]["scale"])
    xs = np.stack([x0] * int(cfg["streams"]))
    behind = []
    for i in layer_order(cfg):
        lc, p = cfg["layers"][i], f"l{i}."
        ml = lc.get("mlp")
        for q in (1, 2) if ml is not None else (1,):
            hc = lambda n: w[f"{p}hc{q}.{n}"]
            h = rms_norm(hyper_read(xs, hc("in")), w[f"{p}norm{q}"], eps)
            h = h + causal_conv(h, w[f"{p}canon{q}"])
            if q == 1:
                y = {"latent_attention": latent_attention, "attention": grouped_attention}[lc["type"]](h, w, p + "mix.", lc["mixer"], eps)
            else:
                y = dense_mlp(h, w, p + "mlp.") if ml["kind"] == "dense" else experts_mlp(h, w, p + "mlp.", ml)
            xs = hyper_write(xs, hc("mix"), hc("out"), y, mult)
        behind.append(xs.sum(axis=0))
    return rms_norm(xs.sum(axis=0), w["final.norm"], eps) @ w["head"].T, behind


# ------------------------------------------------------------------------------------------------ the tests' own configurations, weights and model directories
def rot(dims, base=10000.0, scaling=None):
    r = {"dims": int(dims), "base": float(base)}
    if scaling:
        r["scaling"] = dict(scaling)
    return r


def yarn(factor, original, fast=32.0, slow=1.0):
    return {"factor": float(factor), "original": int(original), "fast": float(fast), "slow": float(slow)}


def dense(ff):
    return {"kind": "dense", "ff": int(ff)}


def moe(experts, top, ff, groups=(1, 1), scale=1.0):
    return {"kind": "moe", "expert": {"ff": int(ff)}, "router": {"experts": int(experts), "top": int(top), "groups": {"count": int(groups[0]), "keep": int(groups[1])}, "scale": float(scale)}}


def latent_layer(heads, dim, rot_dim, vdim, kv_rank, q_rank, rotation=None, scale=None, mlp=None):
    return {"type": "latent_attention", "mlp": mlp, "mixer": {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank, "q_rank": q_rank,
                                                               "rot": rotation or rot(rot_dim), "scale": float(scale if scale is not None else (dim + rot_dim) ** -0.5)}}


def attention_layer(heads, kv_heads, dim, vdim, window, scale=None, mlp=None):
    return {"type": "attention", "mlp": mlp, "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "mask": {"size": int(window)},
                                                        "scale": float(scale if scale is not None else dim ** -0.5)}}


def config(vocab, width, layers, eps=1e-5, taps=3, streams=2, mult=0.5, embed_scale=1.0, loop=None):
    cfg = {"architecture": "Dironex", "vocab": int(vocab), "width": int(width), "norm": {"eps": float(eps)}, "canon": {"taps": int(taps)}, "streams": int(streams),
           "residual_mult": float(mult), "embedding": {"scale": float(embed_scale)}, "layers": layers}
    if loop:
        cfg["loop"] = {"start": int(loop[0]), "stop": int(loop[1]), "times": int(loop[2])}
    return cfg


def bf16_bits(a):
    u = np.ascontiguousarray(a, dtype=np.float32).view(np.uint32).astype(np.uint64)
    return ((u + 0x7FFF + ((u >> 16) & 1)) >> 16).astype(np.uint16)


def to_bf16(a):
    return (bf16_bits(a).astype(np.uint32) << 16).view(np.float32).reshape(np.shape(a))


def weights(cfg, seed):
    """random tensors (bf16-representable f32) for a configuration: products ~ N(0, gain^2 / in), norm weights around 1, every stream fed and read with both signs"""
    rng = np.random.default_rng(seed)
    vocab, width, taps, S = cfg["vocab"], cfg["width"], cfg["canon"]["taps"], cfg["streams"]
    W = {}

    def lin(name, n, k, gain=1.0):
        W[name] = to_bf16(rng.standard_normal((n, k)) * gain / np.sqrt(k))

    def vec(name, n, centre, spread):
        W[name] = to_bf16(centre + spread * (rng.random(n) - 0.5))

    W["embed"] = to_bf16(rng.standard_normal((vocab, width)) / cfg["embedding"]["scale"])
    for i, lc in enumerate(cfg["layers"]):
        p, mx, ml = f"l{i}.", lc["mixer"], lc.get("mlp")
        for q in (1, 2) if ml is not None else (1,):
            vec(f"{p}norm{q}", width, 1.0, 0.6)
            W[f"{p}canon{q}"] = to_bf16(rng.standard_normal((width, taps)) * 0.3)
            vec(f"{p}hc{q}.in", S, 1.0 / S, 1.2), vec(f"{p}hc{q}.out", S, 0.8, 1.6)
            W[f"{p}hc{q}.mix"] = to_bf16(np.eye(S) * 0.9 + 0.25 / S * rng.standard_normal((S, S)))
        m = p + "mix."
        if lc["type"] == "latent_attention":
            H, dim, rd, vd, rank, qr = (mx[k] for k in ("heads", "dim", "rot_dim", "vdim", "kv_rank", "q_rank"))
            lin(m + "dq", qr, width, 2.0), lin(m + "uq", H * (dim + rd), qr, 2.0), lin(m + "dkv", rank + rd, width, 2.0), lin(m + "g", H * vd, width, 1.5)
            vec(m + "dq.norm", qr, 1.0, 0.6), vec(m + "dkv.norm", rank, 1.0, 0.6)
            lin(m + "uk", H * dim, rank, 1.5), lin(m + "uv", H * vd, rank), lin(m + "o", width, H * vd)
        else:
            H, G, dim, vd = (mx[k] for k in ("heads", "kv_heads", "dim", "vdim"))
            lin(m + "q", H * dim, width), lin(m + "k", G * dim, width), lin(m + "v", G * vd, width)
            vec(m + "q.norm", dim, 1.5, 0.6), vec(m + "k.norm", dim, 1.5, 0.6)
            lin(m + "o", width, H * vd)
        f = p + "mlp."
        if ml is None:
            continue
        if ml["kind"] == "dense":
            lin(f + "up", ml["ff"], width, 1.5), lin(f + "down", width, ml["ff"])
            W[f + "act"] = to_bf16(rng.standard_normal(2))
        else:
            E, ff = ml["router"]["experts"], ml["expert"]["ff"]
            lin(f + "router", E, width, 2.0)
            W[f + "correction"] = to_bf16(rng.standard_normal(E) * 0.6 - 0.5)
            for e in range(E):
                lin(f"{f}e{e}.up", ff, width, 1.5), lin(f"{f}e{e}.down", width, ff)
    vec("final.norm", width, 1.0, 0.6)
    lin("head", vocab, width)
    return W


def write_model_dir(path, cfg, W):
    """config.json + model.safetensors (bf16) in the design's layout, written with nothing but the file format"""
    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w", encoding="utf-8") as f:
        json.dump(cfg, f)
    header, blobs, off = {}, [], 0
    for name in sorted(W):
        b = bf16_bits(W[name]).tobytes()
        header[name] = {"dtype": "BF16", "shape": list(np.shape(W[name])), "data_offsets": [off, off + len(b)]}
        blobs.append(b)
        off += len(b)
    head = json.dumps(header).encode()
    with open(os.path.join(path, "model.safetensors"), "wb") as f:
        f.write(len(head).to_bytes(8, "little") + head + b"".join(blobs))


def logit_error(got, want):
    """rms difference per row (means taken off) relative to the rms of the expected logits"""
    a, b = np.asarray(got, dtype=np.float64), np.asarray(want, dtype=np.float64)
    a, b = a - a.mean(-1, keepdims=True), b - b.mean(-1, keepdims=True)
    return np.sqrt(((a - b) ** 2).mean(-1)) / np.sqrt((b ** 2).mean())


def greedy(cfg, W, prompt, n):
    toks, gaps = list(prompt), []
    for _ in range(n):
        row = forward(cfg, W, toks)[0][-1]
        top2 = np.sort(row)[-2:]
        gaps.append(float((top2[1] - top2[0]) / row.std()))
        toks.append(int(row.argmax()))
    return toks[len(prompt):], gaps
