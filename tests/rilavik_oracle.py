"""Rilavik in plain float64 NumPy: every mechanism as one function over a whole sequence, without caches, batches or kernels.  It shares nothing with the product
path (uzu_amd/, csrc/): the tests hold the engine to these equations.

Notation: T positions, d = model width, x [T, d] the residual stream.  Weights are dicts of float64 arrays keyed by the tensor names of a model directory
(linear weights [out, in]); `cfg` is the parsed config.json.
"""
from __future__ import annotations

import json
import os
from typing import Dict, List, Tuple

import numpy as np


def sigmoid(z):
    return 0.5 * (1.0 + np.tanh(0.5 * np.asarray(z, dtype=np.float64)))


def log_sigmoid(z):
    return -np.logaddexp(0.0, -np.asarray(z, dtype=np.float64))


def silu(z):
    return z * sigmoid(z)


def softplus(z):
    return np.logaddexp(0.0, z)


def rms_norm(y, w, eps: float):
    """y [..., n] / sqrt(mean(y^2) + eps) * w"""
    return y / np.sqrt((y ** 2).mean(axis=-1, keepdims=True) + eps) * w


def rms_norm_in_parts(y, w, parts: int, eps: float):
    """y [T, n] cut into `parts` equal consecutive parts, each divided by its own root mean square; the whole times w"""
    T, n = y.shape
    y = y.reshape(T, parts, n // parts)
    return (y / np.sqrt((y ** 2).mean(axis=-1, keepdims=True) + eps)).reshape(T, n) * w


def causal_conv(u, w, bias=None):
    """u [T, C], w [C, taps]: y_t = bias + sum_j w[:, j] u_(t - taps + 1 + j), zeros in front of the sequence (the last tap weighs the current position)"""
    T, C = u.shape
    taps = w.shape[1]
    padded = np.concatenate([np.zeros((taps - 1, C)), u])
    y = sum(w[:, j] * padded[j:j + T] for j in range(taps))
    return y if bias is None else y + bias


def rotate_half(a, dims: int, base: float, factor: float = 1.0, first_position: int = 0):
    """a [T, heads, width]: coordinates (i, i + dims / 2), i < dims / 2, of every head turn by position * base^(-2i / dims) / factor; the rest stay"""
    half = dims // 2
    freq = float(base) ** (-2.0 * np.arange(half) / max(dims, 1)) / factor
    ang = (first_position + np.arange(a.shape[0]))[:, None] * freq[None, :]
    c, s = np.cos(ang)[:, None, :], np.sin(ang)[:, None, :]
    out = a.copy()
    u, v = a[..., :half], a[..., half:dims]
    out[..., :half], out[..., half:dims] = u * c - v * s, v * c + u * s
    return out


def window_attention(q, k, v, scale: float, window: int):
    """q [T, H, dk], k [T, G, dk], v [T, G, dv]; query head a reads key / value head a // (H / G); position i sees j with 0 <= i - j < window (0: every j <= i).  -> [T, H, dv]"""
    T, H, _ = q.shape
    G = k.shape[1]
    dist = np.arange(T)[:, None] - np.arange(T)[None, :]
    seen = (dist >= 0) & ((dist < window) if window else True)
    out = np.zeros((T, H, v.shape[2]))
    for a in range(H):
        g = a // (H // G)
        s = np.where(seen, (q[:, a] @ k[:, g].T) * scale, -np.inf)
        e = np.exp(s - s.max(axis=1, keepdims=True))
        out[:, a] = (e / e.sum(axis=1, keepdims=True)) @ v[:, g]
    return out


def conv_attention_mixer(h, w: Dict[str, np.ndarray], p: str, mx: dict):
    """the left half of the `parallel` mixer: convolved queries, keys and values, rotation, windowed softmax attention, out projection"""
    T = h.shape[0]
    H, G, dk, dv = int(mx["heads"]), int(mx["kv_heads"]), int(mx["dim"]), int(mx["vdim"])
    q, k, v = (causal_conv(h @ w[p + n].T, w[p + n + ".conv"]) for n in ("q", "k", "v"))
    q, k, v = q.reshape(T, H, dk), k.reshape(T, G, dk), v.reshape(T, G, dv)
    rot = mx["rot"]
    turn = lambda a: rotate_half(a, int(rot["dims"]), float(rot["base"]), float((rot.get("scaling") or {}).get("factor", 1.0)))
    o = window_attention(turn(q), turn(k), v, float(mx["scale"]), int(mx["mask"]["size"]))
    return o.reshape(T, H * dv) @ w[p + "o"].T


def decayed_state(q, k, v, decay, state=None):
    """ONE head: q, k [T, N], v [T, dv], decay [T, N] (or [T, 1]); S [N, dv] from `state` (zeros):  S <- decay_t * S (rows) + k_t v_t^T,  o_t = S^T q_t.  -> (o, S)"""
    S = np.zeros((q.shape[1], v.shape[1])) if state is None else state.copy()
    o = np.zeros((q.shape[0], v.shape[1]))
    for t in range(q.shape[0]):
        S = decay[t][:, None] * S + np.outer(k[t], v[t])
        o[t] = S.T @ q[t]
    return o, S


def ssd_mixer(h, w, p: str, mx: dict, eps: float):
    """the right half of the `parallel` mixer: one decay per head and step, keys / queries (B / C) shared by the heads of a group, a step size, a skip, the gate in front of the norm"""
    T = h.shape[0]
    H, dv, N, G = int(mx["heads"]), int(mx["vdim"]), int(mx["state"]), int(mx["groups"])
    inner = H * dv
    z, xbc, dt = np.split(h @ w[p + "in"].T, [inner, 2 * inner + 2 * G * N], axis=1)
    xbc = silu(causal_conv(xbc, w[p + "conv"], w[p + "conv.b"]))
    x, B, C = np.split(xbc, [inner, inner + G * N], axis=1)
    x, B, C = x.reshape(T, H, dv), B.reshape(T, G, N), C.reshape(T, G, N)
    dt = softplus(dt + w[p + "dt_bias"])
    y = np.zeros((T, H, dv))
    for a in range(H):
        g = a // (H // G)
        decay = np.exp(-np.exp(w[p + "A_log"][a]) * dt[:, a])[:, None]
        o, _ = decayed_state(C[:, g], dt[:, a, None] * B[:, g], x[:, a], np.repeat(decay, N, axis=1))
        y[:, a] = o + w[p + "D"][a] * x[:, a]
    y = rms_norm_in_parts(y.reshape(T, inner) * silu(z), w[p + "norm"], int(mx["norm_groups"]), eps)
    return y @ w[p + "o"].T


def parallel_mixer(h, w, p: str, mx: dict, eps: float):
    return float(mx["left_scale"]) * conv_attention_mixer(h, w, p + "left.", mx["left"]) + float(mx["right_scale"]) * ssd_mixer(h, w, p + "right.", mx["right"], eps)


def gla_mixer(h, w, p: str, mx: dict, eps: float):
    """gated linear attention: a decay per head and key channel through a low-rank projection, per-head RMS norm of the read-out, a silu gate"""
    T = h.shape[0]
    H, dk, dv = int(mx["heads"]), int(mx["dim"]), int(mx["vdim"])
    q = (h @ w[p + "q"].T).reshape(T, H, dk) * dk ** -0.5
    k, v = (h @ w[p + "k"].T).reshape(T, H, dk), (h @ w[p + "v"].T).reshape(T, H, dv)
    decay = np.exp(log_sigmoid((h @ w[p + "a1"].T) @ w[p + "a2"].T + w[p + "a2.b"]) / float(mx["tau"])).reshape(T, H, dk)
    o = np.stack([decayed_state(q[:, a], k[:, a], v[:, a], decay[:, a])[0] for a in range(H)], axis=1)
    o = rms_norm(o, w[p + "norm"], eps).reshape(T, H * dv) * silu(h @ w[p + "g"].T)
    return o @ w[p + "o"].T


def moe_mlp(h, w, p: str, ml: dict):
    """sigmoid scores, the `top` largest win (ties: the lower index), not renormalised; a score multiplies its expert's INPUT"""
    top = int(ml["router"]["top"])
    s = sigmoid(h @ w[p + "router"].T)
    chosen = np.argsort(-s, axis=1, kind="stable")[:, :top]
    out = np.zeros_like(h)
    for t in range(h.shape[0]):
        for e in chosen[t]:
            u = s[t, e] * h[t]
            q = f"{p}e{e}."
            out[t] += w[q + "down"] @ (silu(w[q + "gate"] @ u) * (w[q + "up"] @ u))
    return out


def forward(cfg: dict, w: Dict[str, np.ndarray], tokens) -> Tuple[np.ndarray, List[np.ndarray]]:
    """-> (logits [T, vocab], the residual stream behind every layer)"""
    w = {n: np.asarray(a, dtype=np.float64) for n, a in w.items()}
    eps = float(cfg["norm"]["eps"])
    x = w["embed"][np.asarray(tokens, dtype=np.int64)]
    streams = []
    for i, lc in enumerate(cfg["layers"]):
        p = f"l{i}."
        h = rms_norm(x, w[p + "norm1"], eps)
        m = {"parallel": parallel_mixer, "gla": gla_mixer}[lc["type"]](h, w, p + "mix.", lc["mixer"], eps)
        x = x + rms_norm(m, w[p + "norm1b"], eps) * w[p + "ls1"]
        if lc.get("mlp") is not None:
            h = rms_norm(x, w[p + "norm2"], eps)
            x = x + rms_norm(moe_mlp(h, w, p + "mlp.", lc["mlp"]), w[p + "norm2b"], eps) * w[p + "ls2"]
        streams.append(x.copy())
    return rms_norm(x, w["final.norm"], eps) @ w["head"].T, streams


# ------------------------------------------------------------------------------------------------ the tests' own configurations, weights and model directories
def moe(experts, top, ff):
    return {"kind": "moe", "expert": {"ff": int(ff)}, "router": {"experts": int(experts), "top": int(top)}}


def gla_layer(heads, dim, vdim, tau=16.0, rank=3, mlp=None):
    """`rank` (of the decay's two factors) sizes tensors only: kept under '_sizes', which a reader ignores"""
    return {"type": "gla", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "tau": float(tau)}, "mlp": mlp, "_sizes": {"rank": int(rank)}}


def left_half(heads, kv_heads, dim, vdim, window, conv=3, rot_dims=None, base=1e4, factor=None, scale=None):
    rot = {"base": float(base), "dims": int(dim if rot_dims is None else rot_dims)}
    if factor is not None:
        rot["scaling"] = {"factor": float(factor)}
    return {"conv": int(conv), "heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "mask": {"size": int(window)}, "rot": rot,
            "scale": float(scale if scale is not None else dim ** -0.5)}


def right_half(heads, vdim, state, groups=1, norm_groups=1, conv=4):
    return {"conv": int(conv), "heads": heads, "vdim": vdim, "state": state, "groups": groups, "norm_groups": norm_groups}


def parallel_layer(left, right, left_scale=1.0, right_scale=1.0, mlp=None):
    return {"type": "parallel", "mixer": {"left": left, "right": right, "left_scale": float(left_scale), "right_scale": float(right_scale)}, "mlp": mlp}


def config(vocab, width, layers, eps=1e-5):
    return {"architecture": "Rilavik", "vocab": int(vocab), "width": int(width), "norm": {"eps": float(eps)}, "layers": layers}


def bf16_bits(a):
    u = np.ascontiguousarray(a, dtype=np.float32).view(np.uint32).astype(np.uint64)
    return ((u + 0x7FFF + ((u >> 16) & 1)) >> 16).astype(np.uint16)


def to_bf16(a):
    return (bf16_bits(a).astype(np.uint32) << 16).view(np.float32).reshape(np.shape(a))


def weights(cfg, seed):
    """random tensors (bf16-representable f32) for a configuration: products ~ N(0, gain^2 / in), norm weights around 1, decays from fast to slow"""
    rng = np.random.default_rng(seed)
    vocab, width = cfg["vocab"], cfg["width"]
    W = {}

    def lin(name, n, k, gain=1.0):
        W[name] = to_bf16(rng.standard_normal((n, k)) * gain / np.sqrt(k))

    def vec(name, n, centre, spread):
        W[name] = to_bf16(centre + spread * (rng.random(n) - 0.5))

    def taps(name, channels, n):
        W[name] = to_bf16(rng.standard_normal((channels, n)) * 0.4 + np.eye(1, n, n - 1) * 0.6)

    lin("embed", vocab, width, np.sqrt(width))
    for i, lc in enumerate(cfg["layers"]):
        p, mx, ml = f"l{i}.", lc["mixer"], lc.get("mlp")
        for q in (1, 2) if ml is not None else (1,):
            vec(f"{p}norm{q}", width, 1.0, 0.6), vec(f"{p}norm{q}b", width, 1.0, 0.6), vec(f"{p}ls{q}", width, 0.7, 0.6)
        m = p + "mix."
        if lc["type"] == "gla":
            H, dk, dv, rank = mx["heads"], mx["dim"], mx["vdim"], lc["_sizes"]["rank"]
            lin(m + "q", H * dk, width, 1.5), lin(m + "k", H * dk, width, 1.5), lin(m + "v", H * dv, width), lin(m + "g", H * dv, width, 1.5)
            lin(m + "a1", rank, width), lin(m + "a2", H * dk, rank, 2.0), vec(m + "a2.b", H * dk, 1.0, 4.0)
            vec(m + "norm", dv, 1.0, 0.6), lin(m + "o", width, H * dv)
        else:
            L, R, q = mx["left"], mx["right"], m + "left."
            H, G, dk, dv = L["heads"], L["kv_heads"], L["dim"], L["vdim"]
            for n, ch, gain in (("q", H * dk, 2.0), ("k", G * dk, 2.0), ("v", G * dv, 1.0)):
                lin(q + n, ch, width, gain), taps(q + n + ".conv", ch, L["conv"])
            lin(q + "o", width, H * dv)
            H, dv, N, G, q = R["heads"], R["vdim"], R["state"], R["groups"], m + "right."
            inner, mixed = H * dv, H * dv + 2 * G * N
            lin(q + "in", inner + mixed + H, width, 1.5), taps(q + "conv", mixed, R["conv"]), vec(q + "conv.b", mixed, 0.1, 0.6)
            vec(q + "dt_bias", H, -1.5, 3.0), vec(q + "A_log", H, -0.5, 3.0), vec(q + "D", H, 0.5, 1.5), vec(q + "norm", inner, 1.0, 0.6)
            lin(q + "o", width, inner)
        if ml is not None:
            E, ff, f = ml["router"]["experts"], ml["expert"]["ff"], p + "mlp."
            lin(f + "router", E, width, 1.5)
            for e in range(E):
                lin(f"{f}e{e}.gate", ff, width, 2.0), lin(f"{f}e{e}.up", ff, width, 2.0), lin(f"{f}e{e}.down", width, ff)
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
    hj = json.dumps(header).encode()
    hj += b" " * (-len(hj) % 8)
    with open(os.path.join(path, "model.safetensors"), "wb") as f:
        f.write(len(hj).to_bytes(8, "little") + hj + b"".join(blobs))


def logit_error(got, want):
    """per row: RMS over the vocabulary of the difference with its mean taken off, relative to the RMS of the centred expected row"""
    d = np.asarray(got, dtype=np.float64) - np.asarray(want, dtype=np.float64)
    d = d - d.mean(-1, keepdims=True)
    w = np.asarray(want, dtype=np.float64)
    w = w - w.mean(-1, keepdims=True)
    return np.sqrt((d * d).mean(-1)) / np.sqrt((w * w).mean(-1) + 1e-30)


def greedy(cfg, W, prompt, n):
    """n tokens by arg-max, every step a forward pass over the whole sequence"""
    toks = list(prompt)
    for _ in range(n):
        logits, _ = forward(cfg, W, toks)
        toks.append(int(np.argmax(logits[-1])))
    return toks[len(prompt):]
