"""Dironex on the host: identities of the float64 oracle (what the GPU tests lean on), and the config.json reader -- every branch of the schema, the engine
description it produces, its refusals, and what the writer writes read back.  No GPU."""
import json
import os

import numpy as np
import pytest

import dironex_oracle as O
from uzu_amd import desc as D, dironex, loader


def test_oracle_rotation():
    rng = np.random.default_rng(0)
    r = O.rot(8, 1e4)
    x = rng.standard_normal((9, 8))
    y = O.rotate_half(x, np.arange(9), r)
    assert np.allclose(y[0], x[0])  # position 0 turns nothing
    assert np.allclose(x[:, 1] ** 2 + x[:, 5] ** 2, y[:, 1] ** 2 + y[:, 5] ** 2)  # the pair (i, i + 4) keeps its length
    q, k = rng.standard_normal((1, 8)), rng.standard_normal((1, 8))
    s = lambda a, b: float(O.rotate_half(q, [a], r)[0] @ O.rotate_half(k, [b], r)[0])
    assert np.isclose(s(10, 3), s(107, 100))  # scores of rotated queries and keys depend on the distance only
    # scaled frequencies: fast pairs keep theirs, slow pairs are divided by the factor, a ramp between; cos and sin grow with the factor
    f, m = O.rotation_frequencies(32, 1e4, O.yarn(8.0, 512, 32.0, 1.0))
    plain, one = O.rotation_frequencies(32, 1e4, None)
    assert one == 1.0 and m == pytest.approx(0.1 * np.log(8.0) + 1.0)
    ratio = plain / f
    assert ratio[0] == pytest.approx(1.0) and ratio[-1] == pytest.approx(8.0) and np.all(np.diff(ratio) >= -1e-12) and np.any((ratio > 1.01) & (ratio < 7.9))
    empty, _ = O.rotation_frequencies(8, 1e6, O.yarn(2.0, 8, 4.0, 4.0))  # a ramp of no width is a step
    assert set(np.round(O.rotation_frequencies(8, 1e6, None)[0] / empty, 6)) <= {1.0, 2.0}


def test_oracle_hyper_connections_convolution_and_activation():
    rng = np.random.default_rng(1)
    xs, y = rng.standard_normal((3, 5, 4)), rng.standard_normal((5, 4))
    mix = rng.standard_normal((3, 3))
    new = O.hyper_write(xs, mix, np.array([1.0, -2.0, 0.0]), y, 0.5)
    assert np.allclose(new[1], mix[0, 1] * xs[0] + mix[1, 1] * xs[1] + mix[2, 1] * xs[2] - y)  # [from, to]
    assert np.allclose(O.hyper_write(xs[:1], np.eye(1), np.ones(1), y, 0.3)[0], xs[0] + 0.3 * y)  # one copy: the plain residual sum
    assert np.allclose(O.hyper_read(xs, np.array([2.0, 0.0, -1.0])), 2.0 * xs[0] - xs[2])
    h, taps = rng.standard_normal((20, 5)), rng.standard_normal((5, 4))
    c = O.causal_conv(h, taps)
    assert np.allclose(c[0], taps[:, 3] * h[0]) and np.allclose(c[7], sum(taps[:, j] * h[4 + j] for j in range(4)))
    assert np.allclose(O.causal_conv(h, taps[:, 3:]), taps[:, 3] * h)  # one tap: a scale
    z = np.array([-30.0, -1.0, -1e-9, 0.0, 1e-9, 2.0])
    a = O.xielu(z, np.array([0.4, -1.2]))
    sp = lambda v: np.log1p(np.exp(v))
    assert a[3] == 0.0 and a[5] == pytest.approx(sp(0.4) * 4.0 + 1.0) and a[1] == pytest.approx((0.5 + sp(-1.2)) * np.exp(-1.0) - 0.5)
    assert a[0] == pytest.approx((0.5 + sp(-1.2)) * 29.0 - 15.0) and a[2] == pytest.approx(-5e-10, rel=1e-6) and a[4] == pytest.approx(5e-10, rel=1e-6)


def test_oracle_routing():
    w = {"router": np.eye(6), "correction": np.zeros(6)}
    z = lambda *v: np.array([v], dtype=float)
    r = {"experts": 6, "top": 2, "scale": 3.0, "groups": {"count": 3, "keep": 1}}
    # the strongest expert (0) sits in a group that loses on its second best
    ids, wt = O.route(z(3.0, -9.0, 1.0, 2.0, 0.0, 0.0), w, "", r)
    s = 1.0 / (1.0 + np.exp(-np.array([2.0, 1.0])))
    assert list(ids[0]) == [3, 2] and np.allclose(wt[0], 3.0 * s / s.sum())
    # the correction moves the choice and not the weights; negative choice scores of a kept group beat whatever the others have
    w2 = dict(w, correction=np.array([-5.0, -5.0, -5.0, -5.0, -4.0, -4.0]))
    ids, wt = O.route(z(3.0, 3.0, 3.0, 3.0, 0.0, 1.0), w2, "", r)
    assert list(ids[0]) == [5, 4] and wt[0].sum() == pytest.approx(3.0) and wt[0, 0] / wt[0, 1] == pytest.approx(1.0 / (1.0 + np.exp(-1.0)) / 0.5)
    ids, _ = O.route(z(1.0, 0.5, 1.0, 0.5, 1.0, 0.5), w, "", dict(r, groups={"count": 3, "keep": 2}))
    assert list(ids[0]) == [0, 2]  # ties: the lower group, the lower expert


def test_oracle_window_and_latent_cache_identity():
    v = O.causal_window(6, 3)
    assert v.sum() == 1 + 2 + 3 * 4 and v[5, 3] and not v[5, 2] and not v[3, 4]
    assert O.causal_window(6).sum() == 21 and np.array_equal(O.causal_window(6, 1), np.eye(6, dtype=bool))
    # the attention over expanded keys and values equals attention in latent space: q W_uk folded, W_uv behind the weighted sum
    cfg = O.config(vocab=5, width=12, layers=[O.latent_layer(2, 6, 4, 5, 8, 7)])
    W = {k: w.astype(np.float64) for k, w in O.weights(cfg, 3).items()}
    h, mx, p = np.random.default_rng(2).standard_normal((9, 12)), cfg["layers"][0]["mixer"], "l0.mix."
    c = O.rms_norm((h @ W[p + "dkv"].T)[:, :8], W[p + "dkv.norm"], 1e-5)
    kr = O.rotate_half((h @ W[p + "dkv"].T)[:, 8:], np.arange(9), mx["rot"])
    q = (O.rms_norm(h @ W[p + "dq"].T, W[p + "dq.norm"], 1e-5) @ W[p + "uq"].T).reshape(9, 2, 10)
    heads = []
    for a in range(2):
        ql = np.concatenate([q[:, a, :6] @ W[p + "uk"].reshape(2, 6, 8)[a], O.rotate_half(q[:, a, 6:], np.arange(9), mx["rot"])], axis=1)
        ctx = O.softmax_attention(ql @ np.concatenate([c, kr], axis=1).T * mx["scale"], O.causal_window(9), c)
        heads.append(ctx @ W[p + "uv"].reshape(2, 5, 8)[a].T)
    folded = (np.concatenate(heads, axis=1) * O.sigmoid(h @ W[p + "g"].T)) @ W[p + "o"].T
    assert np.allclose(folded, O.latent_attention(h, W, p, mx, 1e-5))


def cfg_full():
    return O.config(vocab=37, width=24, eps=1e-4, taps=3, streams=3, mult=0.4, embed_scale=0.5, loop=(1, 3, 2), layers=[
        O.latent_layer(4, 6, 4, 5, 10, 7, O.rot(4, 500.0, O.yarn(4.0, 128, 16.0, 2.0)), scale=0.3, mlp=O.dense(20)),
        O.attention_layer(6, 3, 4, 8, window=11, scale=0.7, mlp=None),
        O.latent_layer(2, 8, 2, 4, 6, 5, O.rot(2, 1e4), mlp=O.moe(6, 2, 10, (3, 2), 1.5)),
        O.attention_layer(2, 2, 8, 4, window=5, mlp=O.moe(4, 1, 6, (1, 1), 0.5)),
    ])


def test_oracle_is_causal_and_loops():
    cfg = cfg_full()
    W = {k: v.astype(np.float64) for k, v in O.weights(cfg, 2).items()}
    a, behind = O.forward(cfg, W, [3, 1, 4, 1, 5, 9, 2, 6])
    b, _ = O.forward(cfg, W, [3, 1, 4, 1, 5, 9, 7, 7])
    assert np.allclose(a[:6], b[:6]) and not np.allclose(a[6], b[6]) and len(behind) == 6
    assert O.layer_order(cfg) == dironex.layer_runs(cfg) == [0, 1, 2, 1, 2, 3]
    once, _ = O.forward(dict(cfg, loop={"start": 1, "stop": 3, "times": 1}), W, [3, 1, 4])
    assert np.allclose(once, O.forward({k: v for k, v in cfg.items() if k != "loop"}, W, [3, 1, 4])[0])


def write(tmp_path, cfg, W, name="m"):
    O.write_model_dir(str(tmp_path / name), cfg, W)
    return str(tmp_path / name)


def test_reader_maps_every_branch_of_the_schema(tmp_path):
    cfg = cfg_full()
    W = O.weights(cfg, 3)
    b = loader.load_model_dir(write(tmp_path, cfg, W), max_context_length=64)
    assert b.architecture == "Dironex" and b.f32_stream and not b.tied_embeddings and b.vocab_size == 37 and b.model_dim == 24 and b.input_scale == 0.5
    assert b.hyper_streams == 3 and b.residual_mult == pytest.approx(0.4) and b.output_norm.epsilon == 1e-4
    assert [l.weights_of_layer for l in b.layers] == [None, None, None, 1, 2, None]
    la, at, lm, _, _, am = b.layers
    for lw in b.layers:  # a norm in front of a sublayer, its convolution, its connections
        assert lw.pre_mixer_norm.present and lw.pre_mixer_norm.scale_offset == 0.0 and not lw.post_mixer_norm.present and lw.input_conv_taps == 3
        assert lw.input_conv_mixer.shape == (24, 3) and lw.hyper_mixer.shape == (15,)
        assert lw.no_mlp == (lw.hyper_mlp is None) == (lw.input_conv_mlp is None) == (not lw.pre_mlp_norm.present)
    assert np.array_equal(la.hyper_mixer, np.concatenate([W["l0.hc1.in"], W["l0.hc1.out"], W["l0.hc1.mix"].ravel()]))
    # latent attention: query latent | latent + rotated part | gates in one projection
    assert la.mixer_kind == D.MIXER_LATENT_ATTENTION and (la.num_heads, la.head_dim, la.value_head_dim, la.latent_rank, la.latent_rope_dim) == (4, 6, 5, 10, 4)
    assert la.latent_packed and la.has_gate and la.gate_elementwise and la.use_rope and not la.rope_interleaved and la.attention_scale == pytest.approx(0.3)
    assert la.qkv_projection.n == 7 + 10 + 4 + 4 * 5 and np.array_equal(la.qkv_projection.weights[7:21], O.bf16_bits(W["l0.mix.dkv"]))
    assert (la.latent_query_up.n, la.latent_query_up.k) == (4 * 10, 7) and la.latent_query_norm.scales.shape == (7,) and la.latent_norm.scales.shape == (10,)
    r0, r1 = b.ropes[la.rope_index], b.ropes[lm.rope_index]
    assert (r0.kind, r0.head_dim, r0.base, r0.scaling_factor, r0.original_context_length, r0.beta_fast, r0.beta_slow, r0.truncate) == (D.ROPE_YARN, 4, 500.0, 4.0, 128, 16.0, 2.0, True)
    assert (r1.kind, r1.head_dim, r1.base) == (D.ROPE_UNSCALED, 2, 1e4) and len(b.ropes) == 2
    assert la.mlp_plain and la.activation == D.ACT_XIELU and la.hidden_dim == 20 and la.xielu == tuple(float(v) for v in W["l0.mlp.act"])
    # attention: grouped heads, norms per head, no rotation, a window
    assert at.mixer_kind == D.MIXER_ATTENTION and (at.num_heads, at.num_groups, at.head_dim, at.value_head_dim, at.sliding_window_size) == (6, 3, 4, 8, 11)
    assert at.qkv_projection.n == 6 * 4 + 3 * 4 + 3 * 8 and not at.use_rope and not at.has_gate and at.query_norm.scales.shape == (4,) and not at.qk_norm_whole and at.no_mlp
    # experts
    mo = lm.moe
    assert (mo.num_routed_experts, mo.num_active_experts, mo.expert_hidden_dim, mo.routing) == (6, 2, 10, D.MOE_ROUTE_SIGMOID_GROUPS) and mo.plain_experts
    assert (mo.router_groups, mo.router_groups_keep, mo.router_scale) == (3, 2, 1.5) and mo.w13.shape == (6, 10, 24) and mo.w2.shape == (6, 24, 10) and mo.selection_bias.shape == (6,)
    assert np.array_equal(mo.w13[4], O.bf16_bits(W["l2.mlp.e4.up"])) and am.moe.router_groups == 1
    d = b.desc()  # the ctypes description carries them
    assert d.hyper_streams == 3 and d.layers[0].latent_query_rank == 7 and d.layers[0].gate_elementwise == 1 and d.layers[2].moe.plain_experts == 1 and d.layers[2].moe.router_groups_keep == 2
    assert d.layers[0].xielu_q == pytest.approx(float(W["l0.mlp.act"][1])) and d.layers[1].hyper_mlp is None and d.layers[4].weights_of_layer == 3
    assert b.weight_stream_bytes() > 0 and b.prefill_flops(16) > 0 and b.state_bytes_per_token(32) > 0
    spare = dict(W)  # a layer without a feed-forward whose file still carries the second sublayer's tensors: read, not used
    for n in ("norm2", "canon2", "hc2.in", "hc2.out", "hc2.mix"):
        spare["l1." + n] = W["l0." + n]
    assert loader.load_model_dir(write(tmp_path, cfg, spare, "spare"), max_context_length=64).layers[1].no_mlp
    # sizes a configuration leaves to the tensors, one copy without connections, no loop, no groups
    bare = O.config(vocab=37, width=24, streams=1, layers=[O.latent_layer(2, 4, 2, 4, 6, 5, mlp=O.dense(8)), O.attention_layer(2, 2, 4, 4, window=3, mlp=O.moe(3, 1, 4))])
    Wb = {k: v for k, v in O.weights(bare, 1).items() if ".hc" not in k}
    del bare["streams"], bare["layers"][0]["mixer"]["q_rank"], bare["layers"][0]["mlp"]["ff"], bare["layers"][1]["mixer"]["mask"], bare["layers"][1]["mlp"]["router"]["groups"]
    b2 = loader.load_model_dir(write(tmp_path, bare, Wb, "bare"), max_context_length=64)
    assert b2.hyper_streams == 1 and np.array_equal(b2.layers[0].hyper_mixer, np.ones(3)) and b2.layers[0].latent_query_up.k == 5 and b2.layers[0].hidden_dim == 8
    assert b2.layers[1].sliding_window_size == 0 and (b2.layers[1].moe.router_groups, b2.layers[1].moe.router_groups_keep) == (1, 1)


def test_reader_refusals(tmp_path):
    def kind(c, W): c["layers"][1]["type"] = "convolution"
    def mlp(c, W): c["layers"][0]["mlp"]["kind"] = "gated"
    def shape(c, W): W["l1.mix.k"] = W["l1.mix.k"][:-1]
    def extra(c, W): W["l1.mix.extra"] = W["l1.mix.q"]
    def missing(c, W): del W["l0.mix.uq"]
    def no_expert(c, W): del W["l2.mlp.e5.down"]
    def rotation(c, W): c["layers"][0]["mixer"]["rot"]["dims"] = 2
    def no_rotation(c, W): del c["layers"][0]["mixer"]["rot"]
    def heads(c, W): c["layers"][1]["mixer"]["kv_heads"] = 4
    def groups(c, W): c["layers"][2]["mlp"]["router"]["groups"]["count"] = 4
    def keep(c, W): c["layers"][2]["mlp"]["router"]["groups"]["keep"] = 4
    def top(c, W): c["layers"][2]["mlp"]["router"]["top"] = 5
    def width(c, W): c["width"] = 25
    def streams(c, W): c["streams"] = 2
    def taps(c, W): c["canon"]["taps"] = 4
    def loop(c, W): c["loop"]["stop"] = 5
    unsupported = (kind, mlp)
    for i, change in enumerate((kind, mlp, shape, extra, missing, no_expert, rotation, no_rotation, heads, groups, keep, top, width, streams, taps, loop)):
        cfg = cfg_full()
        W = O.weights(cfg, 3)
        change(cfg, W)
        with pytest.raises(loader.UnsupportedModelError if change in unsupported else loader.ModelFormatError):
            loader.load_model_dir(write(tmp_path, cfg, W, f"bad{i}"), max_context_length=64)


def test_what_the_writer_writes_reads_back(tmp_path):
    cfg = dironex.config(37, 16, [
        dironex.latent_attention_layer(2, 8, 4, 6, 12, 10, dironex.rotation(4, 1e4, {"factor": 2.0, "original": 64, "fast": 32.0, "slow": 1.0}), mlp=dironex.moe_mlp(4, 2, 8, 2, 1, 2.5)),
        dironex.attention_layer(2, 1, 8, 4, 9, mlp=dironex.dense_mlp(8))], taps=2, streams=2, residual_mult=0.5, embed_scale=0.25, loop=(0, 1, 2))
    T = dironex.random_tensors(cfg, seed=4)
    dironex.save(str(tmp_path / "w"), cfg, T)
    on_disk = json.load(open(os.path.join(str(tmp_path / "w"), "config.json")))
    assert on_disk["architecture"] == "Dironex"
    b = loader.load_model_dir(str(tmp_path / "w"), max_context_length=32)
    assert len(b.layers) == 3 and b.layers[0].moe.num_active_experts == 2 and b.layers[2].sliding_window_size == 9
    assert np.array_equal(b.embedding.weights, O.bf16_bits(T["embed"]))
    # the oracle reads what the writer wrote
    assert O.forward(on_disk, {k: v.astype(np.float64) for k, v in T.items()}, [1, 2, 3])[0].shape == (3, 37)
