"""Rilavik: a decoder-only design over an f32 residual stream (include/uzu_model_desc.h: ``f32_stream``) with norms on both sides of every sublayer and layer scales, whose
layers mix tokens by windowed attention beside a state-space mixer or by gated linear attention, and whose experts read their input times the router's score; read from its
own ``config.json`` schema.

A model directory holds ``config.json`` (``"architecture": "Rilavik"``) and ``model.safetensors`` (bf16 tensors, linear weights ``[out, in]``).  This module turns it
into the engine's :class:`uzu_amd.desc.ModelBundle` -- the object every other model becomes, so `HipModel`, states, batched steps, sampling and the generate loop are
the engine's own -- and writes such a directory from a configuration and random weights (tests, benchmarks).

The design, in this package's terms (every size comes from ``config.json`` or a tensor's shape, every constant that can differ between models from ``config.json``):

* ``x = embed[token]``; the read-out is ``head`` behind ``final.norm``.  Every norm is an RMS norm with a plain weight (``norm.eps``).
* ``layers[i]``: ``x <- x + ls1 * norm1b(mixer(norm1(x)))``, then (``mlp`` not null) ``x <- x + ls2 * norm2b(mlp(norm2(x)))`` (post_*_norm, layer_scale_*).
* ``type: gla`` (desc.MIXER_GATED_LINEAR_ATTENTION): ``mix.q / k / v / g / a1`` packed into one projection, the decay's second factor ``mix.a2`` (+ ``mix.a2.b``),
  decays ``sigmoid(.)^(1 / tau)`` per head and key channel, the read-out RMS-normed per head (``mix.norm``), times ``silu(g h)``, ``mix.o``.
* ``type: parallel``: ``left_scale * left + right_scale * right`` (``pair_mixer``), both reading the same rows.  ``left`` = attention with ``heads`` query heads on
  ``kv_heads`` key / value heads whose q, k and v pass a causal convolution of ``conv`` taps (``qkv_conv``), rotation of the pairs (i, i + dims / 2) with optionally
  linearly scaled frequencies, causal softmax over the last ``mask.size`` positions.  ``right`` = Mamba-2 (desc.MIXER_STATE_SPACE): ``mix.right.in`` rows
  z | x | B | C | dt, a convolution of ``conv`` taps with bias and silu, ``norm_groups`` norm parts behind the gate.
* ``mlp.kind = moe``: ``router.top`` of ``router.experts`` experts ``down(silu(gate u) * (up u))``, ``u`` = the winner's sigmoid score times the input
  (desc.MOE_ROUTE_SIGMOID_GROUPS with ``router_raw`` and ``weight_on_input``).
"""
from __future__ import annotations

import json
import os
from typing import Dict, List, Optional

import numpy as np

from . import desc as D
from .design_tensors import Tensors as _Tensors, bits_to_f32 as _bits_to_f32, f32_to_bf16_bits as _f32_to_bf16_bits, full_linear as _full

ARCHITECTURE = "Rilavik"


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
    ropes: List[D.RopeConfig] = []

    def rope_index(rot: dict, where: str, at_most: int) -> int:
        dims, sc = int(rot["dims"]), rot.get("scaling")
        if dims % 2 or dims > at_most:
            raise bad(f"config.json: {where}.rot.dims = {dims}: an even number of coordinates, at most dim = {at_most}")
        factor = float(sc["factor"]) if sc else 1.0
        if factor <= 0.0:
            raise bad(f"config.json: {where}.rot.scaling.factor = {factor}")
        r = D.RopeConfig(kind=D.ROPE_LINEAR if sc else D.ROPE_UNSCALED, head_dim=dims, max_sequence_length=max_ctx, base=float(rot["base"]), scaling_factor=factor)
        if r not in ropes:
            ropes.append(r)
        return ropes.index(r)

    vec = lambda n, dim: np.ascontiguousarray(t.f32(n, (dim,)))
    norm = lambda n: D.NormWeights(present=True, epsilon=eps, scales=vec(n, width))
    pack = lambda *parts: _full(np.ascontiguousarray(np.concatenate([t.bits(n, shape) for n, shape in parts], axis=0)))

    def gla(lw: D.LayerWeights, p: str, mx: dict, where: str):
        H, dk, dv, tau = int(mx["heads"]), int(mx["dim"]), int(mx["vdim"]), float(mx["tau"])
        if tau <= 0.0:
            raise bad(f"config.json: {where}.tau = {tau}")
        rank = t.shape(p + "a1")[0]
        lw.mixer_kind, lw.num_heads, lw.num_groups, lw.head_dim, lw.value_head_dim = D.MIXER_GATED_LINEAR_ATTENTION, H, H, dk, dv
        lw.attention_scale, lw.decay_temperature = float(dk) ** -0.5, tau
        lw.qkv_projection = pack((p + "q", (H * dk, width)), (p + "k", (H * dk, width)), (p + "v", (H * dv, width)), (p + "g", (H * dv, width)), (p + "a1", (rank, width)))
        lw.dn_decay_up = _full(t.bits(p + "a2", (H * dk, rank)), np.ascontiguousarray(t.bits(p + "a2.b", (H * dk,))))
        lw.dn_norm_scales, lw.dn_norm_epsilon = vec(p + "norm", dv), eps
        lw.out_projection = _full(t.bits(p + "o", (width, H * dv)))

    def attention(lw: D.LayerWeights, p: str, mx: dict, where: str):
        H, dk, dv = int(mx["heads"]), int(mx["dim"]), int(mx["vdim"])
        G = int(mx.get("kv_heads") or H)
        if H < 1 or G < 1 or H % G:
            raise bad(f"config.json: {where}: {H} heads on {G} kv_heads")
        lw.num_heads, lw.num_groups, lw.head_dim, lw.value_head_dim = H, G, dk, dv
        lw.attention_scale = float(mx["scale"]) if mx.get("scale") is not None else float(dk) ** -0.5
        lw.sliding_window_size = int((mx.get("mask") or {}).get("size") or 0)
        if mx.get("rot") and int(mx["rot"].get("dims") or 0):
            lw.use_rope, lw.rope_index = True, rope_index(mx["rot"], where, dk)
        parts = (("q", H * dk), ("k", G * dk), ("v", G * dv))
        lw.qkv_projection = pack(*[(p + n, (ch, width)) for n, ch in parts])
        if mx.get("conv"):
            lw.qkv_conv = np.ascontiguousarray(np.concatenate([t.f32(f"{p}{n}.conv", (ch, int(mx["conv"]))) for n, ch in parts], axis=0))
        lw.out_projection = _full(t.bits(p + "o", (width, H * dv)))

    def state_space(lw: D.LayerWeights, p: str, mx: dict, where: str):
        H, dv, N, G, parts, taps = int(mx["heads"]), int(mx["vdim"]), int(mx["state"]), int(mx.get("groups") or 1), int(mx.get("norm_groups") or 1), int(mx["conv"])
        inner, mixed = H * dv, H * dv + 2 * G * N
        if H % G or inner % parts:
            raise bad(f"config.json: {where}: {H} heads in {G} groups, {inner} coordinates in {parts} equal norm_groups")
        lw.pair_mixer = D.MIXER_STATE_SPACE
        lw.dn_num_heads, lw.dn_num_groups, lw.dn_head_dim, lw.dn_value_head_dim, lw.dn_kernel_size, lw.dn_norm_epsilon, lw.ssd_norm_groups = H, G, N, dv, taps, eps, parts
        lw.dn_in_proj = _full(t.bits(p + "in", (inner + mixed + H, width)))
        lw.dn_conv_weights, lw.dn_conv_biases = np.ascontiguousarray(t.f32(p + "conv", (mixed, taps))), vec(p + "conv.b", mixed)
        lw.dn_a_log, lw.dn_dt_bias, lw.ssd_skip, lw.dn_norm_scales = vec(p + "A_log", H), vec(p + "dt_bias", H), vec(p + "D", H), vec(p + "norm", inner)
        lw.dn_out_proj = _full(t.bits(p + "o", (width, inner)))

    def experts(lw: D.LayerWeights, p: str, ml: dict, where: str):
        E, top = int(ml["router"]["experts"]), int(ml["router"]["top"])
        ff = int((ml.get("expert") or {}).get("ff") or t.shape(p + "e0.up")[0])
        if not 1 <= top <= E:
            raise bad(f"config.json: {where}: {top} of {E} experts")
        both = lambda e: np.concatenate([t.bits(f"{p}e{e}.up", (ff, width)), t.bits(f"{p}e{e}.gate", (ff, width))], axis=0)
        lw.moe = D.MoeWeights(num_routed_experts=E, num_active_experts=top, expert_hidden_dim=ff, router_weights=t.bits(p + "router", (E, width)), router_biases=None,
                              w13=np.ascontiguousarray(np.stack([both(e) for e in range(E)])), w2=np.ascontiguousarray(np.stack([t.bits(f"{p}e{e}.down", (width, ff)) for e in range(E)])),
                              up_biases=None, down_biases=None, router_renorm=False, routing=D.MOE_ROUTE_SIGMOID_GROUPS, router_raw=True, weight_on_input=True)

    def layer(i: int) -> D.LayerWeights:
        lc = layer_cfgs[i]
        p, kind, mx, ml = f"l{i}.", lc.get("type"), lc.get("mixer") or {}, lc.get("mlp")
        where = f"layers[{i}].mixer"
        lw = D.LayerWeights(mixer_kind=D.MIXER_ATTENTION, hidden_dim=0, activation=D.ACT_SILU, pre_mixer_norm=norm(p + "norm1"), pre_mlp_norm=D.ABSENT_NORM, up_projection=None,
                            down_projection=None, post_mixer_norm=norm(p + "norm1b"), layer_scale_mixer=vec(p + "ls1", width))
        if kind == "gla":
            gla(lw, p + "mix.", mx, where)
        elif kind == "parallel":
            attention(lw, p + "mix.left.", mx.get("left") or {}, where + ".left")
            state_space(lw, p + "mix.right.", mx.get("right") or {}, where + ".right")
            lw.pair_scales = (float(mx.get("left_scale", 1.0)), float(mx.get("right_scale", 1.0)))
        else:
            raise unsupported(f"config.json: layers[{i}].type = {kind!r} (gla | parallel)")
        if ml is None:
            lw.no_mlp = True
            for spare in ("norm2", "norm2b", "ls2"):  # a layer without a feed-forward has no use for them; a file that carries them all the same is read
                if t.has(p + spare):
                    st.consumed.add(p + spare)
        elif ml.get("kind") == "moe":
            lw.pre_mlp_norm, lw.post_mlp_norm, lw.layer_scale_mlp = norm(p + "norm2"), norm(p + "norm2b"), vec(p + "ls2", width)
            experts(lw, p + "mlp.", ml, f"layers[{i}].mlp")
        else:
            raise unsupported(f"config.json: layers[{i}].mlp.kind = {ml.get('kind')!r} (moe, or mlp: null)")
        return lw

    layers = [layer(i) for i in range(len(layer_cfgs))]
    bundle = D.ModelBundle(name=name or os.path.basename(os.path.normpath(path)), vocab_size=int(vocab), model_dim=int(width), max_context_length=max_ctx, rope=D.RopeConfig(),
                           embedding=_full(t.bits("embed", (vocab, width))), output_norm=norm("final.norm"), layers=layers, tied_embeddings=False,
                           output_embedding=_full(t.bits("head", (vocab, width))), ropes=ropes or None, f32_stream=True, architecture=ARCHITECTURE)
    st.assert_all_consumed()
    return bundle


# ------------------------------------------------------------------------------------------------ writer: a configuration + random weights -> a model directory
def random_tensors(cfg: dict, seed: int = 0) -> Dict[str, np.ndarray]:
    """f32 values (already bf16-representable) of every tensor a configuration names, from a seeded generator: linear weights ~ N(0, gain^2 / in), norm weights near 1,
    decays spread between fast and slow"""
    rng = np.random.default_rng(seed)
    rb = lambda a: _bits_to_f32(_f32_to_bf16_bits(np.asarray(a, dtype=np.float32)))
    vocab, width = int(cfg["vocab"]), int(cfg["width"])
    out: Dict[str, np.ndarray] = {}

    def lin(name, n, k, gain=1.0):
        out[name] = rb(rng.standard_normal((n, k), dtype=np.float32) * np.float32(gain / np.sqrt(k)))

    vec = lambda name, n, centre, spread: out.__setitem__(name, rb(centre + spread * (rng.random(n) - 0.5)))
    out["embed"] = rb(rng.standard_normal((vocab, width), dtype=np.float32))
    for i, lc in enumerate(cfg["layers"]):
        p, mx, ml = f"l{i}.", lc["mixer"], lc.get("mlp")
        for s in (1, 2) if ml is not None else (1,):
            vec(f"{p}norm{s}", width, 1.0, 0.4), vec(f"{p}norm{s}b", width, 1.0, 0.4), vec(f"{p}ls{s}", width, 0.5, 0.4)
        m, f = p + "mix.", p + "mlp."
        if lc["type"] == "gla":
            H, dk, dv, rank = int(mx["heads"]), int(mx["dim"]), int(mx["vdim"]), int(mx.get("rank", 16))
            lin(m + "q", H * dk, width), lin(m + "k", H * dk, width), lin(m + "v", H * dv, width), lin(m + "g", H * dv, width)
            lin(m + "a1", rank, width), lin(m + "a2", H * dk, rank), vec(m + "a2.b", H * dk, 1.0, 4.0), vec(m + "norm", dv, 1.0, 0.4), lin(m + "o", width, H * dv)
        else:
            L, R = mx["left"], mx["right"]
            H, G, dk, dv = int(L["heads"]), int(L["kv_heads"]), int(L["dim"]), int(L["vdim"])
            for n, ch in (("q", H * dk), ("k", G * dk), ("v", G * dv)):
                lin(f"{m}left.{n}", ch, width)
                out[f"{m}left.{n}.conv"] = rb(rng.standard_normal((ch, int(L["conv"]))) * 0.5)
            lin(m + "left.o", width, H * dv)
            H, dv, N, G, taps = (int(R[k]) for k in ("heads", "vdim", "state", "groups", "conv"))
            inner, mixed = H * dv, H * dv + 2 * G * N
            lin(m + "right.in", inner + mixed + H, width), lin(m + "right.o", width, inner)
            out[m + "right.conv"] = rb(rng.standard_normal((mixed, taps)) * 0.5)
            vec(m + "right.conv.b", mixed, 0.0, 0.4), vec(m + "right.dt_bias", H, -2.0, 3.0), vec(m + "right.A_log", H, 0.5, 2.0), vec(m + "right.D", H, 0.5, 1.0), vec(m + "right.norm", inner, 1.0, 0.4)
        if ml is None:
            continue
        E, ff = int(ml["router"]["experts"]), int(ml["expert"]["ff"])
        lin(f + "router", E, width)
        for e in range(E):
            lin(f"{f}e{e}.gate", ff, width), lin(f"{f}e{e}.up", ff, width), lin(f"{f}e{e}.down", width, ff)
    vec("final.norm", width, 1.0, 0.4)
    lin("head", vocab, width)
    return out


def save(path: str, cfg: dict, tensors: Dict[str, np.ndarray]):
    """Write config.json + model.safetensors (every tensor as bf16) in this design's layout (`rank` of a gla layer is a size of the writer only: a reader takes it from
    the tensors' shapes)."""
    from .loader import write_safetensors
    os.makedirs(path, exist_ok=True)
    full = json.loads(json.dumps(cfg))
    full["architecture"] = ARCHITECTURE
    for lc in full["layers"]:
        lc["mixer"].pop("rank", None)
    with open(os.path.join(path, "config.json"), "w", encoding="utf-8") as f:
        json.dump(full, f, indent=1, sort_keys=True)
    write_safetensors(os.path.join(path, "model.safetensors"), {k: ("BF16", _f32_to_bf16_bits(v).reshape(np.shape(v))) for k, v in tensors.items()}, {})


def moe_mlp(experts: int, top: int, ff: int) -> dict:
    return {"kind": "moe", "expert": {"ff": int(ff)}, "router": {"experts": int(experts), "top": int(top)}}


def gla_layer(heads: int, dim: int, vdim: int, tau: float = 16.0, rank: int = 16, mlp: Optional[dict] = None) -> dict:
    return {"type": "gla", "mlp": mlp, "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "tau": float(tau), "rank": int(rank)}}


def attention_half(heads: int, kv_heads: int, dim: int, vdim: int, window: int, conv: int = 4, rot_dims: Optional[int] = None, rot_base: float = 10000.0, factor: Optional[float] = None,
                   scale: Optional[float] = None) -> dict:
    rot = {"base": float(rot_base), "dims": int(rot_dims if rot_dims is not None else dim)}
    if factor is not None:
        rot["scaling"] = {"factor": float(factor)}
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": int(conv), "mask": {"size": int(window)}, "rot": rot, "scale": float(scale if scale is not None else dim ** -0.5)}


def state_space_half(heads: int, vdim: int, state: int, groups: int = 1, norm_groups: int = 1, conv: int = 4) -> dict:
    return {"heads": heads, "vdim": vdim, "state": state, "groups": groups, "norm_groups": norm_groups, "conv": int(conv)}


def parallel_layer(left: dict, right: dict, left_scale: float = 1.0, right_scale: float = 1.0, mlp: Optional[dict] = None) -> dict:
    return {"type": "parallel", "mlp": mlp, "mixer": {"left": left, "right": right, "left_scale": float(left_scale), "right_scale": float(right_scale)}}


def config(vocab: int, width: int, layers: List[dict], eps: float = 1e-5) -> dict:
    return {"vocab": int(vocab), "width": int(width), "norm": {"eps": float(eps)}, "layers": layers}
