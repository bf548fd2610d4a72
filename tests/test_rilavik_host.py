"""Rilavik on the host: identities of the float64 oracle (what the GPU tests lean on), and the config.json reader -- every branch of the schema, the engine description it
produces (packed projections, the second mixer's fields, post norms, layer scales), its refusals, and what the writer writes read back.  No GPU."""
import json
import os

import numpy as np
import pytest

import rilavik_oracle as O
from uzu_amd import desc as D, loader, rilavik


def test_oracle_rotation_norms_and_convolution():
    rng = np.random.default_rng(0)
    x = rng.standard_normal((9, 3, 12))
    r = O.rotate_half(x, 8, 1e4, 2.0, first_position=5)
    assert np.allclose(r[..., 8:], x[..., 8:])  # the tail passes unchanged
    assert np.allclose(r[..., 1] ** 2 + r[..., 5] ** 2, x[..., 1] ** 2 + x[..., 5] ** 2)  # a rotation keeps the length of every pair (i, i + dims / 2)
    assert np.allclose(O.rotate_half(x, 8, 1e4)[0], x[0])  # position 0 turns nothing
    assert np.allclose(O.rotate_half(x[:1], 8, 1e4, 4.0, 12), O.rotate_half(x[:1], 8, 1e4, 1.0, 3))  # a factor slows every frequency
    q, k = rng.standard_normal((1, 1, 8)), rng.standard_normal((1, 1, 8))
    s = lambda a, b: float(O.rotate_half(q, 8, 1e4, 8.0, a)[0, 0] @ O.rotate_half(k, 8, 1e4, 8.0, b)[0, 0])
    assert np.isclose(s(10, 3), s(107, 100))  # scores of rotated queries and keys depend on the distance only
    y, w = rng.standard_normal((4, 12)) * np.array([1.0] * 6 + [50.0] * 6), rng.random(12) + 0.5
    n = O.rms_norm_in_parts(y, w, 2, 0.0) / w
    assert np.allclose((n[:, :6] ** 2).mean(-1), 1.0) and np.allclose((n[:, 6:] ** 2).mean(-1), 1.0)
    assert np.allclose(O.rms_norm_in_parts(y, w, 1, 0.3), O.rms_norm(y, w, 0.3)) and np.allclose(O.rms_norm_in_parts(y, w, 12, 0.0), np.sign(y) * w)
    h, taps = rng.standard_normal((20, 5)), rng.standard_normal((5, 4))
    c = O.causal_conv(h, taps)
    assert np.allclose(c[0], taps[:, 3] * h[0]) and np.allclose(c[7], sum(taps[:, j] * h[4 + j] for j in range(4)))
    assert np.allclose(O.causal_conv(h, taps[:, 3:], np.ones(5)), taps[:, 3] * h + 1.0)  # one tap: a scale


def test_oracle_window_attention():
    rng = np.random.default_rng(1)
    q, k, v = rng.standard_normal((20, 4, 6)), rng.standard_normal((20, 2, 6)), rng.standard_normal((20, 2, 3))
    o = O.window_attention(q, k, v, 0.5, 5)
    k2, v2 = k.copy(), v.copy()
    k2[:11], v2[:11] = 7.0, 7.0  # row 15 sees 11 .. 15
    assert np.allclose(O.window_attention(q, k2, v2, 0.5, 5)[15], o[15]) and not np.allclose(O.window_attention(q, k2, v2, 0.5, 6)[15], o[15])
    k2[11], v2[11] = 7.0, 7.0
    assert not np.allclose(O.window_attention(q, k2, v2, 0.5, 5)[15], o[15])
    assert np.allclose(O.window_attention(q, k, v, 0.5, 1), np.repeat(v, 2, axis=1))  # a window of one: the row's own value; heads 0, 1 read group 0
    assert np.allclose(O.window_attention(q, k, v, 0.5, 0), O.window_attention(q, k, v, 0.5, 99))


def test_oracle_decayed_state_is_the_double_sum():
    rng = np.random.default_rng(2)
    T, N, dv = 11, 4, 3
    q, k, v, d = rng.standard_normal((T, N)), rng.standard_normal((T, N)), rng.standard_normal((T, dv)), rng.random((T, N))
    o, S = O.decayed_state(q, k, v, d)
    for i in range(T):  # o_i = sum_(j <= i) <q_i, prod_(j < t <= i) d_t * k_j> v_j
        assert np.allclose(o[i], sum((q[i] * np.prod(d[j + 1:i + 1], axis=0)) @ k[j] * v[j] for j in range(i + 1)))
    a, S1 = O.decayed_state(q[:6], k[:6], v[:6], d[:6])
    b, S2 = O.decayed_state(q[6:], k[6:], v[6:], d[6:], S1)
    assert np.allclose(np.concatenate([a, b]), o) and np.allclose(S2, S)
    one = np.ones((T, N))
    assert np.allclose(O.decayed_state(q, k, v, one)[1], k.T @ v)  # no decay: the plain sum of outer products
    assert np.allclose(O.decayed_state(q, k, v, 0 * one)[0], (q * k).sum(-1, keepdims=True) * v)  # a full decay: the row alone
    assert np.allclose(np.exp(O.log_sigmoid(np.array([-3.0, 0.0, 40.0])) / 1.0), O.sigmoid(np.array([-3.0, 0.0, 40.0])))


def test_oracle_experts_read_their_weighted_input():
    cfg = O.config(vocab=11, width=12, layers=[O.gla_layer(1, 4, 4, mlp=O.moe(4, 1, 6))])
    W = {k: v.astype(np.float64) for k, v in O.weights(cfg, 1).items()}
    h = np.random.default_rng(1).standard_normal((5, 12))
    s = O.sigmoid(h @ W["l0.mlp.router"].T)
    e = s.argmax(1)
    for t in range(5):
        u, p = s[t, e[t]] * h[t], f"l0.mlp.e{e[t]}."
        assert np.allclose(O.moe_mlp(h, W, "l0.mlp.", O.moe(4, 1, 6))[t], W[p + "down"] @ (O.silu(W[p + "gate"] @ u) * (W[p + "up"] @ u)))
    assert not np.allclose(O.moe_mlp(h, W, "l0.mlp.", O.moe(4, 2, 6)), O.moe_mlp(h, W, "l0.mlp.", O.moe(4, 1, 6)))


def cfg_full():
    return O.config(vocab=37, width=24, eps=1e-4, layers=[
        O.parallel_layer(O.left_half(4, 2, 6, 5, 10, conv=3, rot_dims=4, base=500.0, factor=8.0, scale=0.3), O.right_half(6, 4, 5, groups=2, norm_groups=3, conv=2), 0.6, 0.9, mlp=O.moe(4, 2, 10)),
        O.gla_layer(3, 4, 8, tau=12.0, rank=2, mlp=None),
        O.parallel_layer(O.left_half(2, 2, 8, 8, 3, conv=4, base=100.0), O.right_half(2, 4, 6, conv=4), mlp=None),
        O.gla_layer(2, 6, 3, tau=1.0, rank=5, mlp=O.moe(3, 1, 12)),
    ])


def test_oracle_is_causal():
    cfg = cfg_full()
    W = {k: v.astype(np.float64) for k, v in O.weights(cfg, 2).items()}
    a, streams = O.forward(cfg, W, [3, 1, 4, 1, 5, 9, 2, 6])
    b, _ = O.forward(cfg, W, [3, 1, 4, 1, 5, 9, 7, 7])
    assert np.allclose(a[:6], b[:6]) and not np.allclose(a[6], b[6]) and len(streams) == 4


def write(tmp_path, cfg, W, name="m"):
    O.write_model_dir(str(tmp_path / name), cfg, W)
    return str(tmp_path / name)


def test_reader_maps_every_branch_of_the_schema(tmp_path):
    cfg = cfg_full()
    W = O.weights(cfg, 3)
    b = loader.load_model_dir(write(tmp_path, cfg, W), max_context_length=64)
    assert b.architecture == "Rilavik" and b.f32_stream and not b.tied_embeddings and b.vocab_size == 37 and b.model_dim == 24 and b.output_embedding.n == 37
    p, g, c, e = b.layers
    for i, lw in enumerate(b.layers):  # norms on both sides, layer scales
        for n, have in (("norm1", lw.pre_mixer_norm), ("norm1b", lw.post_mixer_norm)):
            assert np.array_equal(have.scales, W[f"l{i}.{n}"]) and have.epsilon == pytest.approx(1e-4)
        assert np.array_equal(lw.layer_scale_mixer, W[f"l{i}.ls1"])
    assert np.array_equal(p.pre_mlp_norm.scales, W["l0.norm2"]) and np.array_equal(p.post_mlp_norm.scales, W["l0.norm2b"]) and np.array_equal(p.layer_scale_mlp, W["l0.ls2"])
    # the pair: convolved windowed attention as the main mixer, the state-space mixer in the dn_* fields
    assert p.mixer_kind == D.MIXER_ATTENTION and p.pair_mixer == D.MIXER_STATE_SPACE and p.pair_scales == (0.6, 0.9) and p.sliding_window_size == 10 and p.attention_scale == pytest.approx(0.3)
    assert (p.num_heads, p.num_groups, p.head_dim, p.value_head_dim) == (4, 2, 6, 5) and p.qkv_projection.n == 4 * 6 + 2 * 6 + 2 * 5 and p.qkv_conv.shape == (46, 3)
    assert np.array_equal(p.qkv_conv[24:36], W["l0.mix.left.k.conv"]) and p.use_rope and b.ropes[p.rope_index].kind == D.ROPE_LINEAR and b.ropes[p.rope_index].scaling_factor == 8.0
    assert b.ropes[p.rope_index].head_dim == 4 and b.ropes[c.rope_index].kind == D.ROPE_UNSCALED and b.ropes[c.rope_index].base == 100.0 and len(b.ropes) == 2
    assert (p.dn_num_heads, p.dn_num_groups, p.dn_head_dim, p.dn_value_head_dim, p.dn_kernel_size, p.ssd_norm_groups) == (6, 2, 5, 4, 2, 3)
    assert p.dn_in_proj.n == 2 * 24 + 2 * 2 * 5 + 6 and p.dn_conv_weights.shape == (44, 2) and p.dn_conv_biases.shape == (44,) and p.dn_norm_scales.shape == (24,) and p.ssd_skip.shape == (6,)
    assert p.dn_norm_epsilon == pytest.approx(1e-4) and c.ssd_norm_groups == 1 and c.dn_num_groups == 1 and c.no_mlp and not c.pre_mlp_norm.present
    # linear attention
    assert g.mixer_kind == D.MIXER_GATED_LINEAR_ATTENTION and (g.num_heads, g.head_dim, g.value_head_dim) == (3, 4, 8) and g.decay_temperature == 12.0 and g.attention_scale == pytest.approx(0.5)
    assert g.qkv_projection.n == 2 * 12 + 2 * 24 + 2 and np.array_equal(g.qkv_projection.weights[48:72], O.bf16_bits(W["l1.mix.g"])) and np.array_equal(g.qkv_projection.weights[72:], O.bf16_bits(W["l1.mix.a1"]))
    assert (g.dn_decay_up.n, g.dn_decay_up.k) == (12, 2) and np.array_equal(g.dn_decay_up.out_biases, O.bf16_bits(W["l1.mix.a2.b"])) and g.dn_norm_scales.shape == (8,) and g.no_mlp
    # experts: raw sigmoid scores on the input, rows [up ; gate]
    mo = p.moe
    assert (mo.num_routed_experts, mo.num_active_experts, mo.expert_hidden_dim, mo.routing) == (4, 2, 10, D.MOE_ROUTE_SIGMOID_GROUPS) and mo.router_raw and mo.weight_on_input and mo.selection_bias is None
    assert np.array_equal(mo.w13[2, 10:], O.bf16_bits(W["l0.mlp.e2.gate"])) and np.array_equal(mo.w13[2, :10], O.bf16_bits(W["l0.mlp.e2.up"])) and mo.w2.shape == (4, 24, 10) and e.moe.num_active_experts == 1
    d = b.desc()  # the ctypes description carries them
    assert d.layers[0].pair_mixer == 1 + D.MIXER_STATE_SPACE and d.layers[0].qkv_conv_taps == 3 and d.layers[0].ssd_norm_groups == 3 and d.layers[1].decay_temperature == 12.0 and d.layers[1].dn_decay_rank == 2
    assert d.layers[0].moe.router_raw == 1 and d.layers[0].moe.weight_on_input == 1 and d.num_ropes == 2
    assert b.weight_stream_bytes() > 0 and b.state_bytes_per_token(50) > 0 and b.prefill_flops(50) > 0
    spare = dict(W)  # a layer without a feed-forward whose file still carries the second sublayer's vectors: read, not used
    for n in ("norm2", "norm2b", "ls2"):
        spare["l1." + n] = W["l0." + n]
    assert loader.load_model_dir(write(tmp_path, cfg, spare, "spare"), max_context_length=64).layers[1].no_mlp


def test_reader_refusals(tmp_path):
    def broken(change, name):
        cfg = cfg_full()
        W = O.weights(cfg, 3)
        change(cfg, W)
        return write(tmp_path, cfg, W, name)

    left, right = (lambda c: c["layers"][0]["mixer"]["left"]), (lambda c: c["layers"][0]["mixer"]["right"])
    def kind(c, W): c["layers"][1]["type"] = "attention"
    def dense(c, W): c["layers"][0]["mlp"]["kind"] = "dense"
    def shape(c, W): W["l0.mix.left.k"] = W["l0.mix.left.k"][:-1]
    def extra(c, W): W["l1.mix.extra"] = W["l1.mix.q"]
    def missing(c, W): del W["l0.mix.right.A_log"]
    def no_scale(c, W): del W["l3.ls2"]
    def odd(c, W): left(c)["rot"]["dims"] = 3
    def wide(c, W): left(c)["rot"]["dims"] = 8
    def factor(c, W): left(c)["rot"]["scaling"]["factor"] = 0.0
    def heads(c, W): left(c)["kv_heads"] = 3
    def groups(c, W): right(c)["groups"] = 4
    def parts(c, W): right(c)["norm_groups"] = 5
    def state(c, W): right(c)["state"] = 6
    def taps(c, W): left(c)["conv"] = 4
    def tau(c, W): c["layers"][1]["mixer"]["tau"] = 0.0
    def top(c, W): c["layers"][0]["mlp"]["router"]["top"] = 5
    def experts(c, W): c["layers"][0]["mlp"]["router"]["experts"] = 5
    def width(c, W): c["width"] = 25
    for i, change in enumerate((kind, dense, shape, extra, missing, no_scale, odd, wide, factor, heads, groups, parts, state, taps, tau, top, experts, width)):
        with pytest.raises(loader.UnsupportedModelError if change in (kind, dense) else loader.ModelFormatError):
            loader.load_model_dir(broken(change, f"bad{i}"), max_context_length=64)


def test_what_the_writer_writes_reads_back(tmp_path):
    cfg = rilavik.config(37, 16, [
        rilavik.parallel_layer(rilavik.attention_half(2, 1, 8, 4, 6, conv=3, rot_dims=4, factor=2.0), rilavik.state_space_half(4, 4, 8, groups=2, norm_groups=2, conv=2), 0.6, 0.9, mlp=rilavik.moe_mlp(3, 1, 8)),
        rilavik.gla_layer(2, 4, 8, tau=8.0, rank=3)], eps=1e-4)
    T = rilavik.random_tensors(cfg, seed=4)
    rilavik.save(str(tmp_path / "w"), cfg, T)
    on_disk = json.load(open(os.path.join(str(tmp_path / "w"), "config.json")))
    assert on_disk["architecture"] == "Rilavik" and "rank" not in on_disk["layers"][1]["mixer"] and "rank" in cfg["layers"][1]["mixer"]
    b = loader.load_model_dir(str(tmp_path / "w"), max_context_length=32)
    assert len(b.layers) == 2 and b.layers[0].pair_mixer == D.MIXER_STATE_SPACE and b.layers[1].dn_decay_up.k == 3 and b.layers[1].decay_temperature == 8.0
    assert np.array_equal(b.embedding.weights, O.bf16_bits(T["embed"]))
    # the oracle reads what the writer wrote
    assert O.forward(on_disk, {k: v.astype(np.float64) for k, v in T.items()}, [1, 2, 3])[0].shape == (3, 37)
