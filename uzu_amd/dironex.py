"""Dironex: a decoder-only design over an f32 residual stream (include/uzu_model_desc.h: ``f32_stream``) that keeps several copies of the stream joined by
hyper-connections, with a causal convolution between every sublayer and its norm, latent attention beside windowed grouped attention, and dense or routed feed-forwards;
read from its own ``config.json`` schema.

A model directory holds ``config.json`` (``"architecture": "Dironex"``) and ``model.safetensors`` (bf16 tensors, linear weights ``[out, in]``).  This module turns it
into the engine's :class:`uzu_amd.desc.ModelBundle` -- the object every other model becomes, so `HipModel`, states, batched steps, sampling and the generate loop are
the engine's own -- and writes such a directory from a configuration and random weights (tests, benchmarks).

The design, in this package's terms (every size comes from ``config.json`` or a tensor's shape, every constant that can differ between models from ``config.json``):

* ``streams`` copies x_a of the row, all ``embed[token] * embedding.scale`` at the start (ModelBundle.hyper_streams).  A sublayer with ``hc*.in / out / mix`` reads
  ``u = sum_a in[a] x_a`` and joins by ``x_b <- sum_a mix[a, b] x_a + residual_mult * out[b] * y`` (LayerWeights.hyper_*); the read-out is ``head`` behind
  ``final.norm`` of the copies' sum.  Without ``streams``: one copy, the plain residual sum.
* a sublayer reads ``h + conv(h)``, ``h = rms(u) * norm*`` (``norm.eps``), ``conv`` = ``canon*``: a causal convolution over positions on every channel, ``canon.taps``
  taps, the last on the current position (LayerWeights.input_conv_*).
* ``loop {start, stop, times}``: layers start .. stop - 1 run ``times`` times with the same tensors; every run has its own sequence state.  The bundle lists layer
  RUNS: a repeated run names the run whose tensors it uses (``weights_of_layer``).
* ``type: latent_attention`` (desc.MIXER_LATENT_ATTENTION): queries through a latent (``mix.dq``, RMS norm ``mix.dq.norm``, ``mix.uq``: heads x [dim | rot_dim]),
  ``mix.dkv`` (``kv_rank`` latent numbers, normed with ``mix.dkv.norm``, + ``rot_dim`` numbers of ONE rotated key part for all heads), per-head keys ``mix.uk`` and
  values ``mix.uv`` of the latent, rotation of the pairs (i, i + dims / 2) with optionally YaRN-scaled frequencies, causal softmax, a sigmoid gate per coordinate of
  the concatenated heads (``mix.g``), ``mix.o``.  ``mix.dq | dkv | g`` are packed into one projection.
* ``type: attention`` (desc.MIXER_ATTENTION): ``heads`` query heads on ``kv_heads`` key / value heads (``mix.q / k / v`` packed, no biases), per-head RMS norm of
  queries and keys, no rotation, causal softmax over the last ``mask.size`` positions, ``mix.o``.
* ``mlp.kind = dense``: ``down(xielu(up h))`` with the two numbers of ``mlp.act``.
* ``mlp.kind = moe``: ``router.top`` of ``router.experts`` experts ``down(max(up h, 0)^2)``, chosen by sigmoid score + ``correction`` among the experts of the
  ``groups.keep`` strongest of ``groups.count`` groups, weighted by the scores over their sum times ``router.scale`` (desc.MOE_ROUTE_SIGMOID_GROUPS).
"""
from __future__ import annotations

import dataclasses
import json
import os
from typing import Dict, List, Optional

import numpy as np

from . import desc as D
from .design_tensors import Tensors as _Tensors, bits_to_f32 as _bits_to_f32, f32_to_bf16_bits as _f32_to_bf16_bits, full_linear as _full

ARCHITECTURE = "Dironex"


def _rope(rot: dict, max_positions: int) -> D.RopeConfig:
    sc = rot.get("scaling")
    if not sc:
        return D.RopeConfig(kind=D.ROPE_UNSCALED, head_dim=int(rot["dims"]), max_sequence_length=max_positions, base=float(rot["base"]))
    return D.RopeConfig(kind=D.ROPE_YARN, head_dim=int(rot["dims"]), max_sequence_length=max_positions, base=float(rot["base"]), scaling_factor=float(sc["factor"]),
                        original_context_length=int(sc["original"]), beta_fast=float(sc["fast"]), beta_slow=float(sc["slow"]), truncate=True)


def layer_runs(cfg: dict) -> List[int]:
    """the layer index of every layer run, in order"""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return list(range(n))
    a, b, times = int(loop["start"]), int(loop["stop"]), int(loop["times"])
    return list(range(a)) + list(range(a, b)) * times + list(range(b, n))


def load(path: str, cfg: dict, st, max_context_length: Optional[int], name: Optional[str], errors) -> D.ModelBundle:
    """config.json (already parsed) + model.safetensors (uzu_amd.loader.SafeTensors) -> ModelBundle.  `errors` = (ModelFormatError, UnsupportedModelError)."""
    bad, unsupported = errors
    t = _Tensors(st, bad)
    vocab, width = t.shape("embed")
    for key, have in (("vocab", vocab), ("width", width)):
        if cfg.get(key) is not None and int(cfg[key]) != have:
            raise bad(f"config.json: {key} = {cfg[key]} but 'embed' is {[vocab, width]}")
    eps = float((cfg.get("norm") or {}).get("eps", 1e-6))
    max_ctx = int(max_context_length or cfg.get("max_context_length") or 4096)
    layer_cfgs = cfg.get("layers")
    if not isinstance(layer_cfgs, list) or not layer_cfgs:
        raise bad("config.json: 'layers' must be a non-empty array")
    loop = cfg.get("loop")
    if loop and not (0 <= int(loop["start"]) < int(loop["stop"]) <= len(layer_cfgs) and int(loop["times"]) >= 1):
        raise bad(f"config.json: loop = {loop}: 0 <= start < stop <= {len(layer_cfgs)} layers, times >= 1")
    taps = int((cfg.get("canon") or {}).get("taps") or 0)
    streams = int(cfg.get("streams") or 0)
    ropes: List[D.RopeConfig] = []

    def rope_index(rot: dict, where: str, dims: int) -> int:
        if int(rot.get("dims") or dims) != dims or dims % 2:
            raise bad(f"config.json: {where}.rot.dims = {rot.get('dims')}: the rotated part's {dims} coordinates, an even number")
        r = _rope(dict(rot, dims=dims), max_ctx)
        if r not in ropes:
            ropes.append(r)
        return ropes.index(r)

    norm = lambda n, dim: D.NormWeights(present=True, epsilon=eps, scales=np.ascontiguousarray(t.f32(n, (dim,))))
    conv = lambda n: np.ascontiguousarray(t.f32(n, (width, taps))) if taps else None
    pack = lambda *parts: _full(np.ascontiguousarray(np.concatenate([t.bits(n, shape) for n, shape in parts], axis=0)))

    def hyper(p: str) -> np.ndarray:
        if not streams:  # one copy: x <- x + residual_mult * y
            return np.ones(3, dtype=np.float32)
        return np.ascontiguousarray(np.concatenate([t.f32(p + "in", (streams,)), t.f32(p + "out", (streams,)), t.f32(p + "mix", (streams, streams)).reshape(-1)]))

    def latent_attention(lw: D.LayerWeights, p: str, mx: dict, where: str):
        H, dim, rd, vd, rank = int(mx["heads"]), int(mx["dim"]), int(mx.get("rot_dim") or 0), int(mx["vdim"]), int(mx["kv_rank"])
        qr = int(mx.get("q_rank") or t.shape(p + "dq")[0])
        lw.mixer_kind, lw.num_heads, lw.num_groups, lw.head_dim, lw.value_head_dim, lw.latent_rank, lw.latent_rope_dim = D.MIXER_LATENT_ATTENTION, H, H, dim, vd, rank, rd
        if rd:
            if not mx.get("rot"):
                raise bad(f"config.json: {where}: rot_dim = {rd} without a rotation")
            lw.use_rope, lw.rope_index = True, rope_index(mx["rot"], where, rd)
        lw.latent_packed = lw.has_gate = lw.gate_elementwise = True
        lw.attention_scale = float(mx["scale"]) if mx.get("scale") is not None else float(dim + rd) ** -0.5
        lw.qkv_projection = pack((p + "dq", (qr, width)), (p + "dkv", (rank + rd, width)), (p + "g", (H * vd, width)))
        lw.latent_query_norm, lw.latent_query_up = norm(p + "dq.norm", qr), _full(t.bits(p + "uq", (H * (dim + rd), qr)))
        lw.latent_norm = norm(p + "dkv.norm", rank)
        lw.latent_up_keys, lw.latent_up_values = _full(t.bits(p + "uk", (H * dim, rank))), _full(t.bits(p + "uv", (H * vd, rank)))
        lw.out_projection = _full(t.bits(p + "o", (width, H * vd)))

    def attention(lw: D.LayerWeights, p: str, mx: dict, where: str):
        H, dim, vd = int(mx["heads"]), int(mx["dim"]), int(mx["vdim"])
        G = int(mx.get("kv_heads") or H)
        if H < 1 or G < 1 or H % G:
            raise bad(f"config.json: {where}: {H} heads on {G} kv_heads")
        lw.num_heads, lw.num_groups, lw.head_dim, lw.value_head_dim = H, G, dim, vd
        lw.attention_scale = float(mx["scale"]) if mx.get("scale") is not None else float(dim) ** -0.5
        lw.sliding_window_size = int((mx.get("mask") or {}).get("size") or 0)
        lw.qkv_projection = pack((p + "q", (H * dim, width)), (p + "k", (G * dim, width)), (p + "v", (G * vd, width)))
        lw.query_norm, lw.key_norm = norm(p + "q.norm", dim), norm(p + "k.norm", dim)
        lw.out_projection = _full(t.bits(p + "o", (width, H * vd)))

    def dense(lw: D.LayerWeights, p: str, ml: dict):
        ff = int(ml.get("ff") or t.shape(p + "up")[0])
        lw.hidden_dim, lw.mlp_plain, lw.activation = ff, True, D.ACT_XIELU
        lw.up_projection, lw.down_projection = _full(t.bits(p + "up", (ff, width))), _full(t.bits(p + "down", (width, ff)))
        lw.xielu = tuple(float(v) for v in t.f32(p + "act", (2,)))

    def experts(lw: D.LayerWeights, p: str, ml: dict, where: str):
        r = ml["router"]
        E, top, ff = int(r["experts"]), int(r["top"]), int((ml.get("expert") or {}).get("ff") or t.shape(p + "e0.up")[0])
        groups = r.get("groups") or {}
        count = int(groups.get("count") or 1)
        keep = int(groups.get("keep") or count)
        if E % count or keep > count or not 1 <= top <= E // count * keep:
            raise bad(f"config.json: {where}: {top} of {E} experts, {keep} of {count} equal groups kept")
        lw.moe = D.MoeWeights(num_routed_experts=E, num_active_experts=top, expert_hidden_dim=ff, router_weights=t.bits(p + "router", (E, width)), router_biases=None,
                              w13=np.ascontiguousarray(np.stack([t.bits(f"{p}e{e}.up", (ff, width)) for e in range(E)])),
                              w2=np.ascontiguousarray(np.stack([t.bits(f"{p}e{e}.down", (width, ff)) for e in range(E)])),
                              up_biases=None, down_biases=None, router_renorm=False, routing=D.MOE_ROUTE_SIGMOID_GROUPS, selection_bias=np.ascontiguousarray(t.f32(p + "correction", (E,))),
                              plain_experts=True, router_groups=count, router_groups_keep=keep, router_scale=float(r.get("scale", 1.0)))

    def layer(i: int) -> D.LayerWeights:
        lc = layer_cfgs[i]
        p, kind, mx, ml = f"l{i}.", lc.get("type"), lc.get("mixer") or {}, lc.get("mlp")
        lw = D.LayerWeights(mixer_kind=D.MIXER_ATTENTION, hidden_dim=0, activation=D.ACT_RELU_SQUARED, pre_mixer_norm=norm(p + "norm1", width), pre_mlp_norm=D.ABSENT_NORM,
                            up_projection=None, down_projection=None, input_conv_taps=taps, input_conv_mixer=conv(p + "canon1"), hyper_mixer=hyper(p + "hc1."))
        if kind == "latent_attention":
            latent_attention(lw, p + "mix.", mx, f"layers[{i}].mixer")
        elif kind == "attention":
            attention(lw, p + "mix.", mx, f"layers[{i}].mixer")
        else:
            raise unsupported(f"config.json: layers[{i}].type = {kind!r} (latent_attention | attention)")
        if ml is None:
            lw.no_mlp = True
            for spare in ("norm2", "canon2", "hc2.in", "hc2.out", "hc2.mix"):  # a layer without a feed-forward has no use for them; a file that carries them all the same is read
                if t.has(p + spare):
                    st.consumed.add(p + spare)
            return lw
        lw.pre_mlp_norm, lw.input_conv_mlp, lw.hyper_mlp = norm(p + "norm2", width), conv(p + "canon2"), hyper(p + "hc2.")
        if ml.get("kind") == "dense":
            dense(lw, p + "mlp.", ml)
        elif ml.get("kind") == "moe":
            experts(lw, p + "mlp.", ml, f"layers[{i}].mlp")
        else:
            raise unsupported(f"config.json: layers[{i}].mlp.kind = {ml.get('kind')!r} (dense | moe, or mlp: null)")
        return lw

    own: Dict[int, int] = {}   # layer index -> its first run
    runs: List[D.LayerWeights] = []
    for i in layer_runs(cfg):
        if i in own:
            runs.append(dataclasses.replace(runs[own[i]], weights_of_layer=own[i]))
            continue
        own[i] = len(runs)
        runs.append(layer(i))
    bundle = D.ModelBundle(name=name or os.path.basename(os.path.normpath(path)), vocab_size=int(vocab), model_dim=int(width), max_context_length=max_ctx, rope=D.RopeConfig(),
                           embedding=_full(t.bits("embed", (vocab, width))), output_norm=norm("final.norm", width), layers=runs, tied_embeddings=False,
                           output_embedding=_full(t.bits("head", (vocab, width))), input_scale=float((cfg.get("embedding") or {}).get("scale", 1.0)), ropes=ropes or None, f32_stream=True,
                           architecture=ARCHITECTURE, hyper_streams=streams or 1, residual_mult=float(cfg.get("residual_mult", 1.0)))
    st.assert_all_consumed()
    return bundle


# ------------------------------------------------------------------------------------------------ writer: a configuration + random weights -> a model directory
def random_tensors(cfg: dict, seed: int = 0) -> Dict[str, np.ndarray]:
    """f32 values (already bf16-representable) of every tensor a configuration names, from a seeded generator: linear weights ~ N(0, gain^2 / in), norm weights near 1,
    hyper-connections near one stream's residual sum spread over the copies"""
    rng = np.random.default_rng(seed)
    rb = lambda a: _bits_to_f32(_f32_to_bf16_bits(np.asarray(a, dtype=np.float32)))
    vocab, width, taps, S = int(cfg["vocab"]), int(cfg["width"]), int(cfg["canon"]["taps"]), int(cfg["streams"])
    out: Dict[str, np.ndarray] = {}

    def lin(name, n, k, gain=1.0):
        out[name] = rb(rng.standard_normal((n, k), dtype=np.float32) * np.float32(gain / np.sqrt(k)))

    vec = lambda name, n, centre, spread: out.__setitem__(name, rb(centre + spread * (rng.random(n) - 0.5)))
    out["embed"] = rb(rng.standard_normal((vocab, width), dtype=np.float32) / np.float32(cfg["embedding"]["scale"]))
    for i, lc in enumerate(cfg["layers"]):
        p, mx, ml = f"l{i}.", lc["mixer"], lc.get("mlp")
        for q in (1, 2) if ml is not None else (1,):
            vec(f"{p}norm{q}", width, 1.0, 0.4)
            out[f"{p}canon{q}"] = rb(rng.standard_normal((width, taps)) * 0.2)
            vec(f"{p}hc{q}.in", S, 1.0 / S, 0.4), vec(f"{p}hc{q}.out", S, 1.0, 0.6)
            out[f"{p}hc{q}.mix"] = rb(np.eye(S) * 0.9 + 0.1 / S * rng.standard_normal((S, S)))
        m, f = p + "mix.", p + "mlp."
        if lc["type"] == "latent_attention":
            H, dim, rd, vd, rank, qr = (int(mx[k]) for k in ("heads", "dim", "rot_dim", "vdim", "kv_rank", "q_rank"))
            lin(m + "dq", qr, width), lin(m + "uq", H * (dim + rd), qr, 1.5), lin(m + "dkv", rank + rd, width), lin(m + "g", H * vd, width)
            vec(m + "dq.norm", qr, 1.0, 0.4), vec(m + "dkv.norm", rank, 1.0, 0.4)
            lin(m + "uk", H * dim, rank, 1.5), lin(m + "uv", H * vd, rank), lin(m + "o", width, H * vd)
        else:
            H, G, dim, vd = (int(mx[k]) for k in ("heads", "kv_heads", "dim", "vdim"))
            lin(m + "q", H * dim, width), lin(m + "k", G * dim, width), lin(m + "v", G * vd, width)
            vec(m + "q.norm", dim, 1.5, 0.6), vec(m + "k.norm", dim, 1.5, 0.6)
            lin(m + "o", width, H * vd)
        if ml is None:
            continue
        if ml["kind"] == "dense":
            lin(f + "up", int(ml["ff"]), width), lin(f + "down", width, int(ml["ff"]))
            vec(f + "act", 2, 0.3, 1.0)
        else:
            E, ff = int(ml["router"]["experts"]), int(ml["expert"]["ff"])
            lin(f + "router", E, width)
            vec(f + "correction", E, 0.0, 0.2)
            for e in range(E):
                lin(f"{f}e{e}.up", ff, width), lin(f"{f}e{e}.down", width, ff)
    vec("final.norm", width, 1.0, 0.4)
    lin("head", vocab, width)
    return out


def save(path: str, cfg: dict, tensors: Dict[str, np.ndarray]):
    """Write config.json + model.safetensors (every tensor as bf16) in this design's layout."""
    from .loader import write_safetensors
    os.makedirs(path, exist_ok=True)
    full = dict(cfg)
    full["architecture"] = ARCHITECTURE
    with open(os.path.join(path, "config.json"), "w", encoding="utf-8") as f:
        json.dump(full, f, indent=1, sort_keys=True)
    write_safetensors(os.path.join(path, "model.safetensors"), {k: ("BF16", _f32_to_bf16_bits(v).reshape(np.shape(v))) for k, v in tensors.items()}, {})


def rotation(dims: int, base: float = 10000.0, scaling: Optional[dict] = None) -> dict:
    r = {"dims": int(dims), "base": float(base)}
    if scaling:
        r["scaling"] = {k: scaling[k] for k in ("factor", "original", "fast", "slow")}
    return r


def dense_mlp(ff: int) -> dict:
    return {"kind": "dense", "ff": int(ff)}


def moe_mlp(experts: int, top: int, ff: int, groups: int = 1, keep: int = 1, scale: float = 1.0) -> dict:
    return {"kind": "moe", "expert": {"ff": int(ff)}, "router": {"experts": int(experts), "top": int(top), "scale": float(scale), "groups": {"count": int(groups), "keep": int(keep)}}}


def latent_attention_layer(heads: int, dim: int, rot_dim: int, vdim: int, kv_rank: int, q_rank: int, rot: dict, scale: Optional[float] = None, mlp: Optional[dict] = None) -> dict:
    return {"type": "latent_attention", "mlp": mlp, "mixer": {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank, "q_rank": q_rank, "rot": rot,
                                                               "scale": float(scale if scale is not None else (dim + rot_dim) ** -0.5)}}


def attention_layer(heads: int, kv_heads: int, dim: int, vdim: int, window: int, scale: Optional[float] = None, mlp: Optional[dict] = None) -> dict:
    return {"type": "attention", "mlp": mlp, "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "mask": {"size": int(window)},
                                                        "scale": float(scale if scale is not None else dim ** -0.5)}}


def config(vocab: int, width: int, layers: List[dict], eps: float = 1e-6, taps: int = 4, streams: int = 4, residual_mult: float = 1.0, embed_scale: float = 1.0,
           loop: Optional[tuple] = None) -> dict:
    cfg = {"vocab": int(vocab), "width": int(width), "norm": {"eps": float(eps)}, "embedding": {"scale": float(embed_scale)}, "layers": layers, "canon": {"taps": int(taps)},
           "streams": int(streams), "residual_mult": float(residual_mult)}
    if loop:
        cfg["loop"] = {"start": int(loop[0]), "stop": int(loop[1]), "times": int(loop[2])}
    return cfg
