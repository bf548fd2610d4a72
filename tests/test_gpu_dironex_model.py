"""Dironex through the engine (HipModel: states, batched steps, prefill / decode, sampling, the generate loops) against the float64 oracle on small models of the
tests' own making: odd sizes, both mixers in any order, dense blocks, experts and neither, looped stretches, one to nine copies of the stream, one to seven
convolution taps, windows of one position up to windows longer than the prompt, expert groups of one expert up to one group of all."""

import dataclasses

import numpy as np
import pytest

import dironex_oracle as O
from uzu_amd import _ffi, loader
from uzu_amd.engine import MODEL_BATCH, MODEL_DEBUG_TAPS, MODEL_FULL_F32, MODEL_NO_GRAPH, HipModel

pytestmark = pytest.mark.gpu

TOL = {True: 4e-5, False: 6e-2}  # full f32 / bf16 products: rms logit error relative to the rms of the logits


def rows_ok(err, full, tol=None):
    """True f32: every row inside the tolerance.  bf16 products: the rounding noise of a narrow stream grows through the layers, and a row whose routing is a close call
    may choose another expert, so nine rows in ten must be inside and the median well inside."""
    err, tol = np.asarray(err), TOL[full] if tol is None else tol
    return bool(err.max() < tol) if full else bool(np.median(err) < tol / 2 and np.mean(err < tol) >= 0.9)


def cfg_a():  # odd sizes: nothing is a multiple of 8, so every kernel runs its general form; three copies, three taps, a loop of two layers
    return O.config(vocab=61, width=36, eps=1e-5, taps=3, streams=3, mult=0.4, embed_scale=0.7, loop=(1, 3, 2), layers=[
        O.latent_layer(3, 10, 6, 7, 13, 9, O.rot(6, 5000.0, O.yarn(3.0, 40, 4.0, 0.5)), scale=0.3, mlp=O.moe(10, 3, 12, (5, 3), 1.7)),
        O.attention_layer(6, 2, 10, 6, window=19, scale=0.35, mlp=None),
        O.latent_layer(2, 5, 2, 9, 7, 11, O.rot(2, 100.0), mlp=O.dense(20)),
        O.attention_layer(2, 2, 7, 5, window=33, mlp=O.moe(4, 2, 10, (2, 1), 0.6)),
    ])


def cfg_b():  # matrix-core friendly sizes: grouped experts, tiled attention, convolution blocks; two copies, four taps
    return O.config(vocab=97, width=64, eps=1e-6, taps=4, streams=2, mult=0.6, embed_scale=0.5, loop=(0, 1, 3), layers=[
        O.attention_layer(4, 2, 16, 16, window=40, scale=0.25, mlp=O.dense(48)),
        O.latent_layer(4, 16, 16, 16, 48, 24, O.rot(16, 500000.0, O.yarn(4.0, 256)), mlp=O.moe(8, 2, 16, (2, 1), 2.0)),
        O.latent_layer(2, 32, 8, 24, 32, 40, O.rot(8), mlp=None),
    ])


def prompt(cfg, n, seed):
    return [int(t) for t in np.random.default_rng(seed).integers(0, cfg["vocab"], size=n)]


def make(hip_ctx, tmp_path, cfg, seed, flags=MODEL_FULL_F32, ctx_len=256, edit=None, name="m"):
    W = O.weights(cfg, seed)
    if edit:
        edit(W)
    O.write_model_dir(str(tmp_path / name), cfg, W)
    W64 = {k: v.astype(np.float64) for k, v in W.items()}
    return W64, HipModel(hip_ctx, loader.load_model_dir(str(tmp_path / name), max_context_length=ctx_len), MODEL_BATCH(2) | MODEL_DEBUG_TAPS | flags)


def in_portions(m, st, toks, cuts):
    """the logits of every position, the tokens brought in portions"""
    assert sum(cuts) == len(toks)
    rows, at = [], 0
    for n in cuts:
        rows.append(m.step_batch([st], [toks[at:at + n]], [list(range(n))])[0])
        at += n
    return np.concatenate(rows)


@pytest.fixture(scope="module")
def models(hip_ctx, tmp_path_factory):
    out = {}
    for name, cfg, seed in (("a", cfg_a(), 11), ("b", cfg_b(), 12)):
        W = O.weights(cfg, seed)
        path = str(tmp_path_factory.mktemp("dironex") / name)
        O.write_model_dir(path, cfg, W)
        bundle = loader.load_model_dir(path, max_context_length=512)
        W64 = {k: v.astype(np.float64) for k, v in W.items()}
        out[name] = (cfg, W64, {full: HipModel(hip_ctx, bundle, MODEL_BATCH(6) | MODEL_DEBUG_TAPS | (MODEL_FULL_F32 if full else 0)) for full in (True, False)})
    yield out
    for _, _, ms in out.values():
        for m in ms.values():
            m.close()


@pytest.mark.parametrize("name", ["a", "b"])
@pytest.mark.parametrize("full", [True, False])
def test_whole_prompt_every_position_and_every_layer_run(models, name, full):
    cfg, W, ms = models[name]
    m = ms[full]
    toks = prompt(cfg, 150, 1)  # positions on both sides of the windows' edges and of the 32-, 64- and 128-key block borders of the attention kernels
    want, behind = O.forward(cfg, W, toks)
    st = m.new_state()
    got, _ = m.step_batch([st], [toks], [list(range(len(toks)))])
    assert len(behind) == m.num_layers
    for l, ref in enumerate(behind):  # the sum of the copies behind every run: names the first one that differs
        err = np.abs(m.read_layer_output_f32(l) - ref).max(-1) / np.abs(ref).max()
        assert rows_ok(err, full, 2e-5 if full else 5e-2), (l, err.max(), np.median(err))
    assert rows_ok(O.logit_error(got, want), full)
    st.close()


def one_layer(layer, vocab=53, width=40, **kw):
    return O.config(vocab=vocab, width=width, layers=[layer], **kw)


LAT = dict(heads=2, dim=8, rot_dim=4, vdim=8, kv_rank=12, q_rank=10)
lat = lambda **kw: O.latent_layer(**{**LAT, **kw})
att = lambda **kw: O.attention_layer(**{**dict(heads=2, kv_heads=1, dim=8, vdim=8, window=21), **kw})
MECHANISMS = {
    "latent_attention": one_layer(lat()),
    "latent_one_head_odd_widths": one_layer(lat(heads=1, dim=5, rot_dim=2, vdim=7, kv_rank=11, q_rank=3)),
    "latent_values_wider_than_keys": one_layer(lat(heads=3, dim=4, rot_dim=6, vdim=20, kv_rank=30, q_rank=17, scale=0.8)),
    "latent_rotation_wider_than_the_plain_part": one_layer(lat(dim=2, rot_dim=24, rotation=O.rot(24, 50.0))),
    "latent_scaled_rotation": one_layer(lat(rot_dim=16, rotation=O.rot(16, 1e4, O.yarn(8.0, 64, 8.0, 0.25)))),
    "latent_scaled_rotation_with_an_empty_ramp": one_layer(lat(rot_dim=8, rotation=O.rot(8, 1e6, O.yarn(2.5, 8, 4.0, 4.0)))),
    "latent_rank_not_a_multiple_of_four": one_layer(lat(kv_rank=14, rot_dim=2)),
    "latent_fragment_across_the_rotated_part": one_layer(lat(kv_rank=12, rot_dim=20, heads=3)),
    "latent_wider_than_the_tiled_core": one_layer(lat(kv_rank=280, q_rank=48)),
    "latent_query_rank_above_a_wave's_registers": one_layer(lat(q_rank=1100)),
    "attention": one_layer(att()),
    "attention_window_of_one_position": one_layer(att(window=1)),
    "attention_window_of_two_positions": one_layer(att(window=2, kv_heads=2)),
    "attention_window_longer_than_the_prompt": one_layer(att(window=500, heads=6, kv_heads=3)),
    "attention_one_head_wide_values": one_layer(att(heads=1, dim=6, vdim=70, window=30)),
    "dense_block": one_layer(att(mlp=O.dense(24))),
    "dense_block_odd": one_layer(lat(mlp=O.dense(19))),
    "experts": one_layer(att(mlp=O.moe(12, 3, 16, (3, 2), 2.5))),
    "experts_one_group": one_layer(att(mlp=O.moe(6, 2, 7, (1, 1), 1.3))),
    "experts_every_group_kept": one_layer(att(mlp=O.moe(8, 3, 8, (4, 4), 1.0))),
    "experts_groups_of_one": one_layer(att(mlp=O.moe(7, 2, 8, (7, 3), 0.5))),
    "experts_all_of_the_kept_group": one_layer(att(mlp=O.moe(9, 3, 8, (3, 1), 1.0))),
    "experts_one_of_many": one_layer(att(mlp=O.moe(70, 1, 5, (10, 4), 3.0))),
    "one_expert": one_layer(att(mlp=O.moe(1, 1, 9, (1, 1), 1.5))),
    "more_experts_than_a_wave": one_layer(att(mlp=O.moe(160, 9, 4, (16, 5), 2.0))),
    "one_copy": one_layer(att(mlp=O.dense(16)), streams=1),
    "four_copies": one_layer(lat(mlp=O.dense(16)), streams=4, mult=1.0),
    "five_copies": one_layer(lat(mlp=O.dense(16)), streams=5, mult=0.2),
    "nine_copies": one_layer(att(mlp=O.dense(16)), streams=9),
    "one_tap": one_layer(lat(mlp=O.dense(16)), taps=1),
    "two_taps": one_layer(lat(mlp=O.dense(16)), taps=2),
    "five_taps": one_layer(lat(mlp=O.dense(16)), taps=5),
    "seven_taps": one_layer(att(mlp=O.dense(16)), taps=7),
    "wide_rows": one_layer(att(mlp=None), width=2112, taps=3),           # a row is more than one step of a workgroup
    "wide_rows_unaligned": one_layer(lat(mlp=O.dense(8)), width=270, taps=5),
    "wide_rows_four_taps_four_copies": one_layer(att(mlp=O.dense(8)), width=1056, taps=4, streams=4),
    "a_loop_of_one_pass": one_layer(lat(mlp=O.dense(16)), loop=(0, 1, 1)),
    "one_layer_five_times": one_layer(att(mlp=O.dense(16), window=9), loop=(0, 1, 5), mult=0.3),
}


@pytest.mark.parametrize("which", sorted(MECHANISMS))
@pytest.mark.parametrize("full", [True, False])
def test_each_mechanism_alone_in_a_one_layer_model(hip_ctx, tmp_path, which, full):
    cfg = MECHANISMS[which]
    W, m = make(hip_ctx, tmp_path, cfg, 5, flags=MODEL_FULL_F32 if full else 0)
    toks = prompt(cfg, 90, 3)
    want, behind = O.forward(cfg, W, toks)
    st = m.new_state()
    got, _ = m.step_batch([st], [toks], [list(range(len(toks)))])
    for l, ref in enumerate(behind):
        assert rows_ok(np.abs(m.read_layer_output_f32(l) - ref).max(-1) / np.abs(ref).max(), full, 2e-5 if full else 5e-2), l
    assert rows_ok(O.logit_error(got, want), full)
    st.reset()  # and token by token from a reused state: the decode forms of the same kernels
    assert rows_ok(O.logit_error(in_portions(m, st, toks[:40], [1] * 40), want[:40]), full)
    st.close()
    m.close()


def test_choice_scores_below_zero_and_groups_that_lose_on_the_second_best(hip_ctx, tmp_path):
    """Every choice score is negative (an expert outside the kept groups counts as minus infinity: at zero it would win), the strongest expert sits in a group whose
    second best is so weak that the group loses, and the weights come from the scores without the correction."""
    cfg = one_layer(att(mlp=O.moe(8, 2, 8, (4, 2), 1.9)))

    def edit(W):
        W["l0.mlp.correction"] = O.to_bf16(np.array([-1.1, -9.0, -2.0, -2.1, -2.2, -2.05, -3.0, -3.1]))
    W, m = make(hip_ctx, tmp_path, cfg, 6, edit=edit)
    toks = prompt(cfg, 80, 5)
    want, _ = O.forward(cfg, W, toks)
    h = np.random.default_rng(2).standard_normal((40, 40))
    ids, weights = O.route(h, W, "l0.mlp.", cfg["layers"][0]["mlp"]["router"])
    assert ids.min() >= 2 and set(ids.ravel()) <= {2, 3, 4, 5} and np.allclose(weights.sum(1), 1.9)
    for flags, full in ((MODEL_FULL_F32, True), (0, False)):
        mm = m if full else make(hip_ctx, tmp_path, cfg, 6, flags=0, edit=edit, name="b")[1]
        st = mm.new_state()
        assert rows_ok(O.logit_error(in_portions(mm, st, toks, [70] + [1] * 10), want), full)
        st.close()
        mm.close()


@pytest.mark.parametrize("full", [True, False])
def test_head_widths_of_real_models_in_both_precisions(hip_ctx, tmp_path, full):
    """The serving precision runs both attention cores on the matrix cores over bf16 caches (the rotated query part turned as it is loaded, key-split decode with a
    merge, the gate in the value product); prompt rows, a portion and decoded tokens against the oracle."""
    cfg = O.config(vocab=97, width=64, taps=4, streams=4, layers=[
        O.latent_layer(4, 128, 64, 128, 192, 96, O.rot(64, 5e5, O.yarn(8.0, 128)), mlp=O.dense(64)),
        O.attention_layer(4, 1, 128, 128, window=100, mlp=O.moe(8, 2, 24, (2, 1), 2.5))])
    W, m = make(hip_ctx, tmp_path, cfg, 13, flags=MODEL_FULL_F32 if full else 0)
    toks = prompt(cfg, 160, 4)
    want, _ = O.forward(cfg, W, toks)
    st = m.new_state()
    assert rows_ok(O.logit_error(in_portions(m, st, toks, [110, 30] + [1] * 20), want), full)
    st.close()
    m.close()


@pytest.mark.parametrize("kv_rank,rot_dim", [(48, 16), (12, 4)])
@pytest.mark.parametrize("full", [True, False])
def test_interleaved_pairs_are_a_permutation_of_the_rotated_coordinates(hip_ctx, tmp_path, full, kv_rank, rot_dim):
    """the engine's other pairing of the rotated coordinates in the attention core's query load: pairs (2i, 2i + 1) over rows brought into that order give the same model"""
    cfg = one_layer(lat(kv_rank=kv_rank, rot_dim=rot_dim))
    W, m = make(hip_ctx, tmp_path, cfg, 5, flags=MODEL_FULL_F32 if full else 0)
    m.close()
    bundle = loader.load_model_dir(str(tmp_path / "m"), max_context_length=256)
    l = bundle.layers[0]
    order = np.arange(rot_dim).reshape(2, rot_dim // 2).T.ravel()  # i, i + rot_dim / 2, i + 1, ...
    up, packed = l.latent_query_up.weights.reshape(l.num_heads, l.head_dim + rot_dim, -1).copy(), l.qkv_projection.weights.copy()
    up[:, l.head_dim:] = up[:, l.head_dim:][:, order]
    lo = l.latent_query_up.k + kv_rank
    packed[lo:lo + rot_dim] = packed[lo:lo + rot_dim][order]
    turned = dataclasses.replace(l, rope_interleaved=True, latent_query_up=dataclasses.replace(l.latent_query_up, weights=np.ascontiguousarray(up.reshape(l.latent_query_up.weights.shape))),
                                 qkv_projection=dataclasses.replace(l.qkv_projection, weights=packed))
    m = HipModel(hip_ctx, dataclasses.replace(bundle, layers=[turned]), MODEL_BATCH(2) | (MODEL_FULL_F32 if full else 0))
    toks = prompt(cfg, 100, 3)
    st = m.new_state()
    assert rows_ok(O.logit_error(in_portions(m, st, toks, [85] + [1] * 15), O.forward(cfg, W, toks)[0]), full)
    st.close()
    m.close()


@pytest.mark.parametrize("name", ["a", "b"])
@pytest.mark.parametrize("full", [True, False])
def test_prefill_then_token_by_token_and_portions_down_to_two_tokens(models, name, full):
    cfg, W, ms = models[name]
    m = ms[full]
    toks = prompt(cfg, 120, 2)
    want, _ = O.forward(cfg, W, toks)
    for cuts in ([100] + [1] * 20, [1] * 30 + [90], [2, 3, 2, 50, 7, 2, 54], [33, 31, 17, 39], [64, 1, 55], [2] * 5 + [110], [7, 7, 2, 16, 32, 56]):
        st = m.new_state()
        got = in_portions(m, st, toks, cuts)
        assert st.context_length == len(toks)
        assert rows_ok(O.logit_error(got, want), full), cuts
        st.close()


@pytest.mark.parametrize("name", ["a", "b"])
def test_unequal_batch_equals_each_request_alone_and_reused_states(models, name):
    cfg, W, ms = models[name]
    m = ms[True]
    reqs = [prompt(cfg, n, 10 + n) for n in (1, 37, 90, 5, 64)]
    head = lambda r: r[:-3] if len(r) > 3 else r
    alone = []
    for r in reqs:
        st = m.new_state()
        rows = [m.step_batch([st], [head(r)], [[len(head(r)) - 1]])[0]]
        rows += [m.step_batch([st], [[t]], [[0]])[0] for t in r[len(head(r)):]]
        alone.append(np.concatenate(rows))
        st.close()
    pool = [m.new_state() for _ in reqs]
    for turn in range(2):  # the second turn reuses the states the first one gave back (reset), in another order: caches and windows of other requests
        states = pool if turn == 0 else pool[::-1]
        lg, _ = m.step_batch(states, [head(r) for r in reqs], [[len(head(r)) - 1] for r in reqs])
        got = [[lg[i]] for i in range(len(reqs))]
        for step in range(3):  # decoded together; the one-token request has left the batch
            live = [i for i, r in enumerate(reqs) if len(r) > 3]
            lg, _ = m.step_batch([states[i] for i in live], [[reqs[i][len(reqs[i]) - 3 + step]] for i in live], [[0]] * len(live))
            for row, i in zip(lg, live):
                got[i].append(row)
        for i in range(len(reqs)):
            assert np.abs(np.stack(got[i]) - alone[i]).max() < 2e-4 * np.abs(alone[i]).max(), (turn, i)
            assert O.logit_error(np.stack(got[i])[-1:], O.forward(cfg, W, reqs[i])[0][-1:]).max() < TOL[True]
        for st in states:
            st.reset()
    for st in pool:
        st.close()


@pytest.mark.parametrize("full", [True, False])
def test_decoding_requests_beside_a_prompt_in_one_pass(models, full):
    """a request that brings one token, one that goes on with two and one that starts with ninety share a pass: rows of one sequence replace their own convolution
    windows, those of several get theirs behind the pass"""
    cfg, W, ms = models["b"]
    m = ms[full]
    a, b, c = prompt(cfg, 45, 31), prompt(cfg, 52, 32), prompt(cfg, 92, 33)
    sa, sb, sc = m.new_state(), m.new_state(), m.new_state()
    m.step_batch([sa, sb], [a[:40], b[:47]], None)
    rows = {0: [], 1: [], 2: []}
    at_a, at_b, at_c = 40, 47, 0
    for na, nb, nc in ((1, 2, 90), (1, 1, 1), (3, 1, 1), ):
        lg, _ = m.step_batch([sa, sb, sc], [a[at_a:at_a + na], b[at_b:at_b + nb], c[at_c:at_c + nc]], [list(range(na)), list(range(nb)), list(range(nc))])
        rows[0].append(lg[:na]), rows[1].append(lg[na:na + nb]), rows[2].append(lg[na + nb:])
        at_a, at_b, at_c = at_a + na, at_b + nb, at_c + nc
    for i, (toks, lo, hi) in enumerate(((a, 40, at_a), (b, 47, at_b), (c, 0, at_c))):
        assert rows_ok(O.logit_error(np.concatenate(rows[i]), O.forward(cfg, W, toks[:hi])[0][lo:hi]), full, TOL[full] if full or i == 2 else 0.12), i
    for st in (sa, sb, sc):
        st.close()


def test_more_requests_than_a_pass_carries_and_prompts_longer_than_a_pass(hip_ctx, tmp_path):
    cfg = O.config(vocab=31, width=16, taps=3, streams=2, layers=[lat(mlp=O.moe(4, 2, 8, (2, 1), 1.0)), att(window=48, mlp=O.dense(8))])
    W, m = make(hip_ctx, tmp_path, cfg, 21, ctx_len=3000)
    reqs = [prompt(cfg, n, n) for n in (9, 2100, 4, 30, 2)]  # 2100 > one pass of 2048 rows; five requests > two per pass
    states = [m.new_state() for _ in reqs]
    lg, sampled = m.step_batch(states, reqs, [[len(r) - 1] for r in reqs], sample=True)
    for i, r in enumerate(reqs):
        want = O.forward(cfg, W, r)[0][-1:]
        assert O.logit_error(lg[i:i + 1], want).max() < (TOL[True] if len(r) < 200 else 2e-4), i
        assert len(r) > 200 or int(sampled[i]) == int(np.argmax(want))
        assert states[i].context_length == len(r)
    st = m.new_state()  # the long prompt: against the same prompt through two explicit portions
    m.step_batch([st], [reqs[1][:1500]], [[]])
    two, _ = m.step_batch([st], [reqs[1][1500:]], [[599]])
    assert np.abs(two[0] - lg[1]).max() < 2e-4 * np.abs(two).max()
    m.close()


@pytest.mark.parametrize("full", [True, False])
def test_long_decoding(models, full):
    cfg, W, ms = models["b"]
    m = ms[full]
    toks = prompt(cfg, 230, 5)
    want, _ = O.forward(cfg, W, toks)
    st = m.new_state()
    got = in_portions(m, st, toks, [10] + [1] * 220)  # 220 decoded tokens over the windows' edges and the key blocks' borders
    assert rows_ok(O.logit_error(got, want), full)
    st.close()


def look_alikes(W, pairs, keys, values, canon=0.02):
    """What layer 0 reads is made (nearly) its own token's row, the `keys` projections read the first half of it and the `values` projections the second; the two tokens
    of a pair share the first half of their rows and have opposite second halves: one's query points at the other's key, where another value stands."""
    half = W["embed"].shape[1] // 2
    for a, b in pairs:
        W["embed"][b, :half], W["embed"][b, half:] = W["embed"][a, :half], -W["embed"][a, half:]  # (equal norms)
    W["l0.canon1"] = O.to_bf16(W["l0.canon1"] * canon)
    for n in keys:
        W[n][:, half:] = 0.0
    for n in values:
        W[n][:, :half] = 0.0


@pytest.mark.parametrize("full", [True, False])
def test_a_far_key_among_hundreds_decides_the_logits(hip_ctx, tmp_path, full):
    """The last token of a 700-token prompt looks like the token at position 2 and like no other, and queries are made the keys of their own token (the query latent is
    the key latent, the query's plain part the head's key): that one far key shares the softmax with the row itself.  Replacing it must move the last logits exactly
    as the oracle says, in a whole prompt and when the tail is decoded -- a key that is dropped, doubled, or read from a neighbouring row shows."""
    cfg = O.config(vocab=42, width=32, taps=2, streams=2, layers=[O.latent_layer(2, 16, 8, 8, 24, 12, O.rot(8, 1e5, O.yarn(4.0, 100)), scale=4.0)])

    def match(W):
        # the first 12 latent numbers carry the keys, the last 12 the values
        dkv, uk, uv = W["l0.mix.dkv"], W["l0.mix.uk"], W["l0.mix.uv"]
        dkv[:12, 16:], dkv[12:24, :16], uk[:], uv[:, :12], W["l0.mix.dkv.norm"][:12] = 0.0, 0.0, 0.0, 0.0, 1.0
        uk.reshape(2, 16, 24)[:, :12, :12] = np.eye(12)
        W["l0.mix.dq"], W["l0.mix.dq.norm"] = dkv[:12].copy(), np.ones(12, dtype=np.float32)
        uq = W["l0.mix.uq"].reshape(2, 24, 12).copy()
        uq[:, :16], uq[:, 16:] = uk[:, :12].reshape(2, 16, 12), uq[:, 16:] * 0.05
        W["l0.mix.uq"] = O.to_bf16(uq.reshape(48, 12))
        look_alikes(W, [(39, 41)], (), ())
    W, m = make(hip_ctx, tmp_path, cfg, 8, flags=MODEL_FULL_F32 if full else 0, ctx_len=1024, edit=match)
    base = [int(t) for t in np.random.default_rng(4).integers(0, 39, size=700)]  # tokens 39, 40 and 41 are kept for the marked positions
    base[2], base[-1] = 39, 41
    other = list(base)
    other[2] = 40
    want = [O.forward(cfg, W, t)[0][-1] for t in (base, other)]
    assert O.logit_error(want[0][None], want[1][None]).max() > 0.15, "the oracle itself does not see the token"
    for toks, ref in zip((base, other), want):
        st = m.new_state()
        whole, _ = m.step_batch([st], [toks], [[699]])
        st.reset()
        m.step_batch([st], [toks[:640]], [[]])
        for t in toks[640:-1]:
            m.step_batch([st], [[t]], [[]])
        dec, _ = m.step_batch([st], [[toks[-1]]], [[0]])
        assert O.logit_error(whole, ref[None]).max() < TOL[full] and O.logit_error(dec, ref[None]).max() < TOL[full]
        st.close()
    m.close()


@pytest.mark.parametrize("window", [1, 5, 32, 33, 64, 130])
@pytest.mark.parametrize("full", [True, False])
def test_keys_just_inside_and_just_outside_a_window(hip_ctx, tmp_path, window, full):
    """Queries are made the keys of their own token, so a marked token's query points at its look-alike: once at distance window - 1 (the last position the row sees) and
    once at distance window (the first it does not).  Every position of a prompt, portions cut at, in front of and behind these places, and decoded tokens are held to
    the oracle; the oracle itself tells a window that is off by one."""
    layer = lambda size: O.attention_layer(2, 1, 16, 8, window=size, scale=0.5)
    cfg = O.config(vocab=41, width=32, taps=2, streams=2, layers=[layer(window)])

    def match(W):
        look_alikes(W, [(37, 38), (39, 40)], ("l0.mix.k",), ("l0.mix.v",))
        W["l0.mix.q"] = np.concatenate([W["l0.mix.k"]] * 2)
        W["l0.mix.q.norm"] = W["l0.mix.k.norm"].copy()
    W, m = make(hip_ctx, tmp_path, cfg, 8, flags=MODEL_FULL_F32 if full else 0, ctx_len=512, edit=match)
    n = 2 * window + 40
    toks = [int(t) for t in np.random.default_rng(6).integers(0, 37, size=n)]
    inside, outside = n - 20, n - 7
    toks[inside - (window - 1)], toks[inside] = 37, 38
    toks[outside - window], toks[outside] = 39, 40
    want, _ = O.forward(cfg, W, toks)
    for size in {window - 1, window + 1} - {0}:
        off = O.forward(dict(cfg, layers=[layer(size)]), W, toks)[0]
        row = inside if size < window else outside
        assert O.logit_error(off[row:row + 1], want[row:row + 1]).max() > 0.15, size
    for cuts in ([n], [n - 30] + [1] * 30, [inside, 1, n - inside - 1], [inside - 1, 2, n - inside - 1], [outside - window, window, n - outside], [outside - window + 1, window, n - outside - 1]):
        st = m.new_state()
        err = O.logit_error(in_portions(m, st, toks, [c for c in cuts if c]), want)
        assert rows_ok(err, full), cuts
        assert max(err[inside], err[outside]) < TOL[full], cuts
        st.close()
    m.close()


def test_the_convolution_window_carries_every_tap_across_cuts(hip_ctx, tmp_path):
    """Taps that grow with the distance: what lies taps - 1 positions back weighs most.  Cut at every place of a short prompt, the row behind the cut takes that input
    from the state: for the mixer and the feed-forward, on a state another request has just left."""
    cfg = O.config(vocab=41, width=32, taps=4, streams=3, layers=[att(mlp=O.dense(16)), lat(mlp=O.moe(4, 1, 8, (2, 1), 1.0))])

    def far(W):
        for n in W:
            if "canon" in n:
                W[n] = O.to_bf16(W[n] * np.array([8.0, 2.0, 0.5, 0.1]))
    W, m = make(hip_ctx, tmp_path, cfg, 9, edit=far)
    toks = prompt(cfg, 12, 2)
    want, _ = O.forward(cfg, W, toks)
    near = {k: (v * (np.arange(4) > 0) if "canon" in k else v) for k, v in W.items()}
    assert O.logit_error(O.forward(cfg, near, toks)[0][5:], want[5:]).min() > 0.05
    st = m.new_state()
    for cut in range(1, 11):
        st.reset()
        m.step_batch([st], [prompt(cfg, 20, 40 + cut)], [[]])
        st.reset()
        assert O.logit_error(in_portions(m, st, toks, [cut, 12 - cut]), want).max() < TOL[True], cut
    st.close()
    m.close()


def test_the_first_tokens_and_a_state_that_held_another_request(models):
    """Positions 0, 1, 2 of a sequence: zeros in front of every convolution, one-key softmaxes -- also on a state that another, longer request has just left (reset):
    nothing of it may be read."""
    cfg, W, ms = models["a"]
    m = ms[True]
    st = m.new_state()
    m.step_batch([st], [prompt(cfg, 80, 9)], [[]])
    for n, seed in ((1, 1), (2, 2), (3, 3)):
        st.reset()
        toks = prompt(cfg, n, seed)
        got, _ = m.step_batch([st], [toks], [list(range(n))])
        assert O.logit_error(got, O.forward(cfg, W, toks)[0]).max() < TOL[True]
    st.reset()
    toks = prompt(cfg, 4, 7)
    assert O.logit_error(in_portions(m, st, toks, [1] * 4), O.forward(cfg, W, toks)[0]).max() < TOL[True]
    st.close()


@pytest.mark.parametrize("name", ["a", "b"])
def test_greedy_generation_through_prefill_and_decode(models, name):
    """The engine's own entry points: HipModel.prefill + chained decode (the sampled token is fed back on the device), then the stochastic sampler's plumbing."""
    cfg, W, ms = models[name]
    m = ms[True]
    p = prompt(cfg, 25, 7)
    want, gaps = O.greedy(cfg, W, p, 10)
    assert min(gaps) > 1e-3, "the oracle's own greedy stream has a near tie: pick another seed"
    m.reset()
    m.set_sampling(None)
    got = [int(m.prefill(np.asarray(p, dtype=np.uint32)))] + [int(t) for t in m.decode(9)[0]]
    assert got == want and m.context_length == len(p) + 9
    assert np.argmax(m.read_logits_f32()) == want[-1]
    m.reset()
    m.set_sampling(seed=3, temperature=1e-4)  # temperature -> 0 of the stochastic sampler is greedy
    assert [int(m.prefill(np.asarray(p, dtype=np.uint32)))] + [int(t) for t in m.decode(4)[0]] == want[:5]
    m.set_sampling(None)
    m.reset()


def test_generate_loop_of_the_text_front_end_and_the_pool(hip_ctx, tmp_path):
    """LanguageModel.generate on a directory without tokenizer.json, and SequencePool.generate: prompts of unequal length prefilled in one batch and decoded
    together, requests leaving as they finish (one by a stop token), their states reused by a second call -- against each prompt generated alone by the oracle"""
    from uzu_amd.language_model import LanguageModel
    from uzu_amd.serving import SequencePool
    cfg = cfg_a()
    W = O.weights(cfg, 31)
    O.write_model_dir(str(tmp_path / "g"), cfg, W)
    W64 = {k: v.astype(np.float64) for k, v in W.items()}
    p = prompt(cfg, 12, 3)
    prompts = {"x": prompt(cfg, 3, 41), "y": prompt(cfg, 40, 42), "z": prompt(cfg, 17, 43)}
    streams = {k: O.greedy(cfg, W64, q, n) for k, q, n in (("p", p, 11), *((k, q, 8) for k, q in prompts.items()))}
    assert min(min(g) for _, g in streams.values()) > 1e-3, "a near tie in the oracle's greedy streams: pick another seed"
    lm = LanguageModel(hip_ctx, str(tmp_path / "g"), max_context_length=128, flags=MODEL_FULL_F32, tokenizer_required=False)
    res = lm.generate(p, max_tokens=11, chunk=4)
    assert res.token_ids == streams["p"][0] and res.prompt_tokens == 12
    lm.close()
    m = HipModel(hip_ctx, loader.load_model_dir(str(tmp_path / "g"), max_context_length=128), MODEL_BATCH(4) | MODEL_FULL_F32)
    stop = streams["y"][0][4]
    cut = lambda seq: seq[:seq.index(stop)] if stop in seq else seq
    pool = SequencePool(m)
    for _ in range(2):
        got = pool.generate(prompts, max_tokens=8, stop_token_ids=[stop])
        assert got == {k: cut(streams[k][0]) for k in prompts}
        assert not pool.live and len(pool.free) == 3
    pool.close()
    m.close()


@pytest.mark.parametrize("full", [True, False])
def test_decode_graph_replays_equal_plain_launches(hip_ctx, tmp_path, full):
    """The chained decode step is ONE captured hipGraph per state that reads its position from device memory.  Replayed in several calls, with eager batched steps of
    OTHER states (which overwrite the model's pass tables) and synchronisations between them, every token and the logits after every call must equal those of a
    model that decodes with plain launches."""
    cfg = cfg_b()
    O.write_model_dir(str(tmp_path / "m"), cfg, O.weights(cfg, 77))
    bundle = loader.load_model_dir(str(tmp_path / "m"), max_context_length=256)
    base = MODEL_BATCH(4) | (MODEL_FULL_F32 if full else 0)
    graph, plain = HipModel(hip_ctx, bundle, base), HipModel(hip_ctx, bundle, base | MODEL_NO_GRAPH)
    p, other = prompt(cfg, 70, 8), prompt(cfg, 33, 9)
    firsts = [m.prefill(np.asarray(p, dtype=np.uint32)) for m in (graph, plain)]
    assert firsts[0] == firsts[1]
    side = [m.new_state() for m in (graph, plain)]
    for call in range(4):
        toks = [m.decode(5)[0] for m in (graph, plain)]
        assert list(toks[0]) == list(toks[1]), call
        assert np.array_equal(graph.read_logits_f32(), plain.read_logits_f32()), call
        for m, st in zip((graph, plain), side):  # eager work on another state between the replays
            m.step_batch([st], [other[call * 8:(call + 1) * 8]], [[7]])
    assert graph.context_length == 70 + 20
    for m in (graph, plain):
        m.close()


def test_a_copied_state_goes_on_like_its_source(models):
    cfg, W, ms = models["a"]
    m = ms[True]
    toks = prompt(cfg, 50, 15)
    src, dst = m.new_state(), m.new_state()
    m.step_batch([src], [toks[:41]], [[]])
    dst.copy_from(src)
    m.step_batch([src], [prompt(cfg, 9, 16)], [[]])  # the source goes another way
    assert O.logit_error(in_portions(m, dst, toks[41:], [1, 2, 6]), O.forward(cfg, W, toks)[0][41:]).max() < TOL[True]
    src.close(), dst.close()


@pytest.mark.parametrize("full", [True, False])
def test_convolution_behind_a_norm_without_connections(hip_ctx, tmp_path, full):
    """The same layers on a single stream without hyper-connections (the plain residual sum of the engine's other designs): the normed rows pass the convolution kernels
    of their own -- against the one-copy model with identity connections."""
    cfg = O.config(vocab=53, width=40, streams=1, mult=1.0, layers=[lat(mlp=O.dense(16)), att(mlp=O.moe(6, 2, 8, (3, 2), 1.5)), att(mlp=None)])

    def identity(W):
        for n in W:
            if ".hc" in n:
                W[n] = np.ones_like(W[n])
    W = O.weights(cfg, 4)
    identity(W)
    O.write_model_dir(str(tmp_path / "m"), cfg, W)
    bundle = loader.load_model_dir(str(tmp_path / "m"), max_context_length=256)
    single = dataclasses.replace(bundle, hyper_streams=0, layers=[dataclasses.replace(l, hyper_mixer=None, hyper_mlp=None) for l in bundle.layers])
    toks = prompt(cfg, 100, 3)
    want, behind = O.forward(cfg, {k: v.astype(np.float64) for k, v in W.items()}, toks)
    for b in (bundle, single):
        m = HipModel(hip_ctx, b, MODEL_BATCH(2) | MODEL_DEBUG_TAPS | (MODEL_FULL_F32 if full else 0))
        st = m.new_state()
        got = in_portions(m, st, toks, [80, 2, 8] + [1] * 10)
        assert rows_ok(O.logit_error(got, want), full)
        assert rows_ok(np.abs(m.read_layer_output_f32(2) - behind[2][-1:]).max(-1) / np.abs(behind[2]).max(), full, 2e-5 if full else 5e-2)
        st.close()
        m.close()


def test_refusals_of_the_engine(hip_ctx, tmp_path):
    """what the engine does not run it refuses at creation, by name"""
    cfg = cfg_b()
    O.write_model_dir(str(tmp_path / "m"), cfg, O.weights(cfg, 3))
    bundle = loader.load_model_dir(str(tmp_path / "m"), max_context_length=64)
    last = len(bundle.layers) - 1
    def changed(at, **kw):
        return dataclasses.replace(bundle, layers=[dataclasses.replace(l, **kw) if i == at else l for i, l in enumerate(bundle.layers)])
    absent = dataclasses.replace(bundle.layers[0].pre_mixer_norm, present=False)
    for broken, why in ((changed(last, hyper_mixer=None), "in | out | mix"), (changed(last, pre_mixer_norm=absent), "undivided RMS norm"),
                        (changed(last, post_mixer_norm=bundle.layers[0].pre_mixer_norm), "belong to a single stream"), (changed(last, latent_packed=False), "packed projection"),
                        (changed(last - 1, moe=dataclasses.replace(bundle.layers[last - 1].moe, router_groups=3)), "equal groups"),
                        (changed(last - 1, moe=dataclasses.replace(bundle.layers[last - 1].moe, num_active_experts=5)), "equal groups"),
                        (dataclasses.replace(bundle, hyper_streams=17), "hyper-connections")):
        with pytest.raises(_ffi.UzuHipError, match=why.replace("|", r"\|")):
            HipModel(hip_ctx, broken, MODEL_FULL_F32)
    with pytest.raises(_ffi.UzuHipError):  # the mechanisms belong to the f32-stream designs
        HipModel(hip_ctx, dataclasses.replace(bundle, f32_stream=False), 0)


def random_config(seed):
    """a configuration drawn at random: sizes, head counts, layer order, loop, constants"""
    rng = np.random.default_rng(seed)
    pick = lambda *xs: xs[int(rng.integers(len(xs)))]
    layers = []
    for _ in range(int(rng.integers(2, 6))):
        count, size = pick(1, 2, 4), pick(2, 3, 4)
        keep = int(rng.integers(1, count + 1))
        mlp = pick(None, O.dense(pick(16, 40, 72)), O.moe(count * size, int(rng.integers(1, keep * size + 1)), pick(8, 16, 24), (count, keep), pick(0.5, 1.0, 2.5)))
        if pick("attention", "latent") == "attention":
            G = pick(1, 2, 3)
            layers.append(O.attention_layer(G * pick(1, 2, 4), G, pick(8, 16, 24, 64), pick(8, 16, 24), window=pick(1, 7, 32, 65, 200), scale=pick(0.1, 0.2, 0.35), mlp=mlp))
        else:
            rd = pick(2, 8, 16, 32)
            scaling = pick(None, O.yarn(pick(1.5, 4.0, 16.0), pick(16, 100, 4096), pick(8.0, 32.0), pick(0.5, 1.0)))
            layers.append(O.latent_layer(pick(1, 2, 3, 4), pick(8, 16, 24, 40), rd, pick(8, 16, 24), pick(8, 16, 40, 64), pick(5, 16, 32), O.rot(rd, pick(1e3, 1e4, 5e5), scaling),
                                         scale=pick(0.1, 0.2, 0.35), mlp=mlp))
    n = len(layers)
    a = int(rng.integers(0, n))
    loop = pick(None, (a, int(rng.integers(a + 1, n + 1)), pick(1, 2, 3)))
    return O.config(vocab=pick(50, 257, 640), width=pick(24, 40, 64, 96, 122), layers=layers, eps=pick(1e-6, 1e-5, 1e-3), taps=pick(1, 2, 3, 4, 6), streams=pick(1, 2, 3, 4, 6),
                    mult=pick(0.2, 0.5, 1.0), embed_scale=pick(0.5, 1.0, 4.0), loop=loop)


@pytest.mark.parametrize("seed", range(10))
def test_configurations_drawn_at_random(hip_ctx, tmp_path, seed):
    """whole prompt, prompt + decoded tail and an unequal batch on a configuration nobody chose, in both precisions"""
    cfg = random_config(100 + seed)
    W = O.weights(cfg, seed)
    O.write_model_dir(str(tmp_path / "m"), cfg, W)
    W64 = {k: v.astype(np.float64) for k, v in W.items()}
    bundle = loader.load_model_dir(str(tmp_path / "m"), max_context_length=400)
    a, b = prompt(cfg, 170, seed), prompt(cfg, 45, seed + 50)
    want_a, want_b = O.forward(cfg, W64, a)[0], O.forward(cfg, W64, b)[0]
    for full in (True, False):
        m = HipModel(hip_ctx, bundle, MODEL_BATCH(3) | (MODEL_FULL_F32 if full else 0))
        st = m.new_state()
        whole, _ = m.step_batch([st], [a], [list(range(170))])
        st.reset()
        cut = in_portions(m, st, a, [130] + [1] * 40)
        st2 = m.new_state()
        st.reset()
        both, _ = m.step_batch([st2, st], [b, a[:100]], [list(range(45)), list(range(100))])
        for got, want in ((whole, want_a), (cut, want_a), (both[:45], want_b), (both[45:], want_a[:100])):
            err = O.logit_error(got, want)
            assert (err.max() < 1e-4 and np.median(err) < 1e-5) if full else (np.median(err) < 3e-2 and np.mean(err < 8e-2) >= 0.9), (cfg, full, err.max(), np.median(err))
        m.close()
