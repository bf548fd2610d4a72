"""The two recurrences and the gated norm of the Rilavik design alone: the HIP kernels behind their one-sequence C entries (csrc/capi_stream32.hip) against the float64
oracle, and the forms of one kernel against each other -- decays from 'nearly one' to 'gone in a step', channels of both kinds side by side, chunk and block borders, rows
whose packed columns sit on and off 16-byte borders, state widths from one to beyond a slab and a tile."""
import ctypes as C

import numpy as np
import pytest

import rilavik_oracle as O
from uzu_amd import _ffi

pytestmark = pytest.mark.gpu
u32, f32c = C.c_uint32, C.c_float


def ptr(a):
    return None if a is None else a.ctypes.data_as(C.c_void_p)


def f32(a):
    return np.ascontiguousarray(a, dtype=np.float32)


def channel_state(ctx, q, k, v, pre, tau, state, start, form, q_scale=1.0, pad=0):
    """a decay per head and key channel: q, k, pre [T, H, dim], v [T, H, vdim], state [H, dim, vdim]"""
    T, H, dim = q.shape
    vd = v.shape[2]
    out, st = np.empty((T, H * vd), dtype=np.float32), f32(state).copy()
    _ffi.call("uzu_hip_s32_decayed_state", ctx._h, ptr(f32(q)), ptr(f32(k)), ptr(f32(v)), ptr(f32(pre)), u32(0), f32c(tau), None, None, None, f32c(q_scale), ptr(st), ptr(out), u32(T), u32(start),
              u32(H), u32(H), u32(dim), u32(vd), u32(form), u32(pad))
    return out.reshape(T, H, vd), st


def head_state(ctx, q, k, v, pre, a_log, dt_bias, skip, state, start, form, pad=0):
    """one decay per head: q, k [T, G, dim], v [T, H, vdim], pre [T, H]"""
    T, G, dim = q.shape
    H, vd = v.shape[1:]
    out, st = np.empty((T, H * vd), dtype=np.float32), f32(state).copy()
    _ffi.call("uzu_hip_s32_decayed_state", ctx._h, ptr(f32(q)), ptr(f32(k)), ptr(f32(v)), ptr(f32(pre)), u32(1), f32c(0.0), ptr(f32(a_log)), ptr(f32(dt_bias)), None if skip is None else ptr(f32(skip)),
              f32c(1.0), ptr(st), ptr(out), u32(T), u32(start), u32(H), u32(G), u32(dim), u32(vd), u32(form), u32(pad))
    return out.reshape(T, H, vd), st


def want_channel(q, k, v, pre, tau, state, q_scale=1.0):
    decay = np.exp(O.log_sigmoid(pre) / tau)
    o, S = zip(*[O.decayed_state(q[:, a] * q_scale, k[:, a], v[:, a], decay[:, a], state[a]) for a in range(q.shape[1])])
    return np.stack(o, axis=1), np.stack(S)


def want_head(q, k, v, pre, a_log, dt_bias, skip, state):
    H, G = v.shape[1], q.shape[1]
    dt = O.softplus(pre + dt_bias)
    o, S = [], []
    for a in range(H):
        g = a // (H // G)
        decay = np.repeat(np.exp(-np.exp(a_log[a]) * dt[:, a])[:, None], q.shape[2], axis=1)
        oo, ss = O.decayed_state(q[:, g], dt[:, a, None] * k[:, g], v[:, a], decay, state[a])
        o.append(oo + (skip[a] * v[:, a] if skip is not None else 0.0)), S.append(ss)
    return np.stack(o, axis=1), np.stack(S)


def close(got, want, tol=5e-6):
    """[.., head, .., values]: against the largest number of the head (rows of a result may cancel)"""
    got, want = np.asarray(got, dtype=np.float64), np.asarray(want)
    scale = np.abs(want).max(axis=-1, keepdims=True)
    scale = np.maximum(scale, 0.2 * scale.max(axis=0 if want.shape[0] > 1 else -1, keepdims=True))
    return float((np.abs(got - want) / (scale + 1e-30)).max()) < tol


CHANNEL = [  # rows, start, heads, dim, vdim, tau, pad
    (1, 0, 2, 3, 5, 1.0, 0), (1, 7, 3, 48, 32, 16.0, 0), (5, 0, 1, 1, 1, 2.0, 0), (16, 3, 2, 16, 16, 16.0, 1), (63, 0, 2, 32, 64, 16.0, 0), (64, 0, 2, 33, 65, 4.0, 3), (65, 9, 3, 64, 128, 16.0, 0),
    (129, 1, 2, 100, 24, 1.0, 2), (200, 64, 2, 128, 128, 16.0, 0), (257, 0, 1, 130, 200, 8.0, 0), (90, 5, 1, 260, 20, 16.0, 0), (70, 2, 1, 513, 7, 16.0, 1), (66, 1, 1, 1024, 8, 16.0, 0), (640, 0, 2, 40, 72, 16.0, 0),
]


@pytest.mark.parametrize("case", CHANNEL)
def test_decay_per_channel_both_forms_against_the_recurrence(hip_ctx, case):
    T, start, H, dim, vd, tau, pad = case
    rng = np.random.default_rng(T + dim)
    q, k, v = rng.standard_normal((T, H, dim)), rng.standard_normal((T, H, dim)), rng.standard_normal((T, H, vd))
    pre = rng.standard_normal((T, H, dim)) * 4.0 + np.where(rng.random((1, H, dim)) < 0.5, 6.0, -6.0)  # channels that keep and channels that forget, side by side
    pre[rng.random(pre.shape) < 0.02] = -90.0  # and a step that wipes a channel (tau permitting)
    state = rng.standard_normal((H, dim, vd))
    r = lambda *a: [f32(x).astype(np.float64) for x in a]  # the oracle sees the f32 inputs
    q, k, v, pre, state = r(q, k, v, pre, state)
    want, S = want_channel(q, k, v, pre, tau, state if start else 0 * state, 0.25)
    for form in (1, 2, 0):
        got, st = channel_state(hip_ctx, q, k, v, pre, tau, state, start, form, 0.25, pad)
        assert close(got, want) and close(st, S), form


HEAD = [  # rows, start, heads, groups, dim, vdim, pad
    (1, 0, 2, 1, 3, 5, 0), (1, 9, 4, 2, 32, 32, 0), (7, 0, 3, 3, 8, 4, 1), (16, 2, 2, 1, 16, 64, 0), (63, 0, 4, 2, 32, 32, 0), (64, 5, 2, 2, 128, 64, 0), (65, 0, 4, 1, 31, 63, 2), (130, 1, 2, 1, 128, 128, 0),
    (200, 3, 3, 1, 66, 100, 1), (300, 0, 2, 2, 256, 64, 0), (100, 4, 1, 1, 12, 300, 0), (640, 0, 4, 2, 64, 64, 0), (70, 1, 1, 1, 1, 1, 0),
]


@pytest.mark.parametrize("case", HEAD)
def test_decay_per_head_with_step_and_skip_both_forms_against_the_recurrence(hip_ctx, case):
    T, start, H, G, dim, vd, pad = case
    rng = np.random.default_rng(T + dim)
    q, k, v = rng.standard_normal((T, G, dim)), rng.standard_normal((T, G, dim)), rng.standard_normal((T, H, vd))
    pre = rng.standard_normal((T, H)) * 3.0
    a_log, dt_bias, skip = rng.uniform(-3.0, 3.0, H), rng.uniform(-6.0, 1.0, H), rng.standard_normal(H)  # rates from 1 / 20 to 20 per unit step
    state = rng.standard_normal((H, dim, vd))
    q, k, v, pre, a_log, dt_bias, skip, state = (f32(x).astype(np.float64) for x in (q, k, v, pre, a_log, dt_bias, skip, state))
    for sk in (skip, None):
        want, S = want_head(q, k, v, pre, a_log, dt_bias, sk, state if start else 0 * state)
        for form in (1, 2, 0):
            got, st = head_state(hip_ctx, q, k, v, pre, a_log, dt_bias, sk, state, start, form, pad)
            assert close(got, want) and close(st, S), (form, sk is None)


@pytest.mark.parametrize("form", [1, 2])
def test_a_quiet_stretch_behind_a_storm_keeps_its_digits(hip_ctx, form):
    """Forty steps whose decays multiply to e^-2000 and then steps that hardly decay: what the quiet rows see of each other must not suffer from the storm in front of
    them (a difference of running sums would lose four digits here)."""
    T, dim, vd = 64, 32, 32
    rng = np.random.default_rng(1)
    q, k, v = (f32(rng.standard_normal((T, 1, n))).astype(np.float64) for n in (dim, dim, vd))
    pre = np.full((T, 1), -4.0)
    pre[:40] = 50.0
    pre = f32(pre).astype(np.float64)
    a_log, dt_bias = np.zeros(1), np.zeros(1)
    zero = np.zeros((1, dim, vd))
    want, _ = want_head(q, k, v, pre, a_log, dt_bias, None, zero)
    got, _ = head_state(hip_ctx, q, k, v, pre, a_log, dt_bias, None, zero, 0, form)
    assert close(got[45:], want[45:], 2e-6)
    cp = f32(np.broadcast_to(np.where(np.arange(T)[:, None, None] < 40, -50.0, 5.0), (T, 1, dim))).astype(np.float64)
    want, _ = want_channel(q, k, v, cp, 1.0, zero)
    got, _ = channel_state(hip_ctx, q, k, v, cp, 1.0, zero, 0, form)
    assert close(got[45:], want[45:], 2e-6)


@pytest.mark.parametrize("form", [1, 2])
def test_a_far_key_reaches_the_last_row_through_the_state_alone(hip_ctx, form):
    """500 rows, keys and queries orthogonal but for one pair: row 3's key is the last row's query.  The last result is that one value times the decay of everything in
    between -- a block, a chunk or a carried decay left out or applied twice shows as a factor."""
    T, dim, vd = 500, 16, 8
    rng = np.random.default_rng(2)
    q, k = np.zeros((T, 1, dim)), np.zeros((T, 1, dim))
    k[:, 0, 1:] = rng.standard_normal((T, dim - 1))
    q[:, 0, 1:] = rng.standard_normal((T, dim - 1))
    k[3, 0], q[-1, 0] = np.eye(dim)[0], np.eye(dim)[0]
    v = f32(rng.standard_normal((T, 1, vd))).astype(np.float64)
    pre = f32(rng.uniform(2.0, 4.0, (T, 1, dim))).astype(np.float64)
    q, k = f32(q).astype(np.float64), f32(k).astype(np.float64)
    zero = np.zeros((1, dim, vd))
    got, _ = channel_state(hip_ctx, q, k, v, pre, 16.0, zero, 0, form)
    expect = v[3, 0] * np.exp((O.log_sigmoid(pre[4:, 0, 0]) / 16.0).sum())
    assert np.abs(got[-1, 0] - expect).max() < 2e-5 * np.abs(expect).max()
    pre = f32(rng.uniform(-6.0, -4.0, (T, 1))).astype(np.float64)
    got, _ = head_state(hip_ctx, q, k, v, pre, np.zeros(1), np.zeros(1), None, zero, 0, form)
    dt = O.softplus(pre[:, 0])
    expect = dt[3] * v[3, 0] * np.exp(-dt[4:].sum())
    assert np.abs(got[-1, 0] - expect).max() < 2e-5 * np.abs(expect).max()


def test_portions_through_the_carried_state_equal_the_whole(hip_ctx):
    T, H, dim, vd = 300, 2, 24, 40
    rng = np.random.default_rng(3)
    q, k, v, pre = (f32(rng.standard_normal((T, H, n))) for n in (dim, dim, vd, dim))
    zero = np.zeros((H, dim, vd), dtype=np.float32)
    whole, S = channel_state(hip_ctx, q, k, v, pre, 16.0, zero, 0, 0)
    for cuts in ([2, 62, 64, 1, 171], [128, 172], [1] * 5 + [295], [17, 16, 267]):
        st, at, rows = zero, 0, []
        for n in cuts:
            o, st = channel_state(hip_ctx, q[at:at + n], k[at:at + n], v[at:at + n], pre[at:at + n], 16.0, st, at, 0)
            rows.append(o)
            at += n
        assert close(np.concatenate(rows), whole.astype(np.float64)) and close(st, S.astype(np.float64)), cuts


@pytest.mark.parametrize("shape", [(1, 128, 2), (3, 7, 7), (2, 96, 1), (5, 1000, 4), (70, 2048, 2), (1, 4100, 1)])
def test_gated_norm_in_parts(hip_ctx, shape):
    rows, width, parts = shape
    rng = np.random.default_rng(width)
    y, g, w = f32(rng.standard_normal((rows, width)) * rng.uniform(0.1, 20.0, (1, width))), f32(rng.standard_normal((rows, width)) * 3.0), f32(rng.random(width) + 0.5)
    out = np.empty((rows, width), dtype=np.float32)
    _ffi.call("uzu_hip_s32_gated_norm", hip_ctx._h, ptr(y), ptr(g), ptr(w), ptr(out), f32c(1e-4), f32c(0.7), u32(rows), u32(width), u32(parts))
    want = 0.7 * O.rms_norm_in_parts(y.astype(np.float64) * O.silu(g.astype(np.float64)), w.astype(np.float64), parts, 1e-4)
    assert np.abs(out - want).max() < 3e-6 * np.abs(want).max()
