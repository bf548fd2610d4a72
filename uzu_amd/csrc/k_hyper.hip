// k_hyper.hip -- hyper-connections of the f32-stream designs (kernels_stream32.h: HyperStepParams): the residual stream is `streams` copies of the row; between two
// sublayers stands one launch that joins the first one's result to the copies, reads the row of the second one from them, norms it and (a pass of one row per
// sequence) runs its input convolution.
//
// A column's copies meet at that column only, so a thread takes its columns' copies into registers, forms the new copies from the old ones and writes them in
// place.  The row's sum of squares is folded in a fixed order: a row's result does not depend on what else the pass carries.
#include "device_utils.h"
#include "kernels_stream32.h"

namespace uzu {
namespace k {

namespace {

template <int V> struct Cols {
    float v[V];
};
template <int V> __device__ __forceinline__ Cols<V> ldc(const float* p) {
    Cols<V> r;
    if (V == 4) {
        const f32x4_v t = *(const f32x4_v*)p;
#pragma unroll
        for (int i = 0; i < V; ++i) r.v[i] = t[i];
    } else {
        r.v[0] = p[0];
    }
    return r;
}
template <int V> __device__ __forceinline__ void stc(float* p, const Cols<V>& a) {
    if (V == 4) {
        f32x4_v t;
#pragma unroll
        for (int i = 0; i < V; ++i) t[i] = a.v[i];
        *(f32x4_v*)p = t;
    } else {
        p[0] = a.v[0];
    }
}

constexpr int kTapsAhead = 4; // an input convolution of at most that many taps has its weights and window loaded in front of the row's sum of squares

// the mixing weights of a launch (the same for every thread)
template <int SM> struct Mix {
    float in[SM], out[SM], mix[SM][SM];
    __device__ __forceinline__ explicit Mix(const HyperStepParams& p) {
        const uint32_t S = p.streams;
#pragma unroll
        for (int a = 0; a < SM; ++a) {
            const bool on = (uint32_t)a < S;
            in[a] = on ? (p.read ? p.read[a] : 1.0f) : 0.0f;
            out[a] = on && p.y ? p.mult * p.join[S + a] : 0.0f;
#pragma unroll
            for (int b = 0; b < SM; ++b) mix[a][b] = on && (uint32_t)b < S && p.y ? p.join[2 * S + a * S + b] : 0.0f;
        }
    }
};

// columns c .. c + V - 1 of stream row `src`: the old copies and the sublayer's result
template <int SM, int V> struct Copies {
    Cols<V> x[SM], y;
    __device__ __forceinline__ Copies(const HyperStepParams& p, uint32_t src, uint32_t c) {
        const size_t at = (size_t)src * p.d + c;
#pragma unroll
        for (int a = 0; a < SM; ++a)
            if ((uint32_t)a < p.streams) x[a] = ldc<V>(p.src + a * p.src_stride + at);
        if (p.y) y = ldc<V>(p.y + at);
    }
};
// joins the result, stores the new copies (and their sum), returns what the next sublayer reads
template <int SM, int V> __device__ __forceinline__ Cols<V> join_and_read(const HyperStepParams& p, const Mix<SM>& m, const Copies<SM, V>& old, uint32_t src, uint32_t c) {
    const uint32_t S = p.streams;
    const size_t at = (size_t)src * p.d + c;
    Cols<V> u, sum;
#pragma unroll
    for (int i = 0; i < V; ++i) u.v[i] = sum.v[i] = 0.0f;
#pragma unroll
    for (int b = 0; b < SM; ++b) {
        if ((uint32_t)b >= S) continue;
        Cols<V> now = old.x[b];
        if (p.y) {
#pragma unroll
            for (int i = 0; i < V; ++i) {
                float v = 0.0f;
#pragma unroll
                for (int a = 0; a < SM; ++a)
                    if ((uint32_t)a < S) v = fmaf(m.mix[a][b], old.x[a].v[i], v);
                now.v[i] = fmaf(m.out[b], old.y.v[i], v);
            }
            if (p.dst) stc<V>(p.dst + b * p.dst_stride + at, now);
        }
#pragma unroll
        for (int i = 0; i < V; ++i) u.v[i] = fmaf(m.in[b], now.v[i], u.v[i]), sum.v[i] += now.v[i];
    }
    if (p.sum_out) stc<V>(p.sum_out + at, sum);
    return u;
}

// A workgroup of NT threads per row.  SM: most copies (p.streams <= SM); V: columns per thread and step (4 where rows are 16-byte aligned, else 1).
// ONE: a row is one step (d <= NT V): it stays in registers, and what the norm and the convolution need is on its way while the sum of squares is taken.
template <int SM, int V, int NT, bool ONE>
__global__ void __launch_bounds__(NT) hyper_step_kernel(HyperStepParams p) {
    extern __shared__ float s_u[]; // [d], not ONE: what the sublayer reads, in front of its norm (a thread reads back its own columns only)
    __shared__ float s_red[NT / 64];
    const uint32_t r = blockIdx.x, src = p.row_index ? p.row_index[r] : r, tid = threadIdx.x, d = p.d;
    const bool conv = p.conv_w && p.taps > 1;
    const uint32_t z = conv ? p.row_seq[r] : 0;
    float* window = nullptr; // the one row of its sequence with an input convolution: the carried window; entries in front of position 0 count as zeros
    uint32_t t = 0;
    auto find_window = [&]() {
        if (conv) t = p.spans[z].start, window = p.states[z] + p.state_offset;
    };
    Cols<V> u1, sc1, win1[kTapsAhead];
    float w1[V * kTapsAhead];
    const bool ahead = ONE && p.conv_w && p.taps <= kTapsAhead;
    float ss = 0.0f;
    if (ONE) {
        const uint32_t c = tid * V;
        if (c < d) {
            const Copies<SM, V> old(p, src, c);
            if (p.h) sc1 = ldc<V>(p.scales + c);
            if (ahead && V == 4 && p.taps == 4 && kTapsAhead == 4) {
#pragma unroll
                for (int i = 0; i < V; ++i) {
                    const f32x4_v w = *(const f32x4_v*)(p.conv_w + ((size_t)c + i) * 4);
#pragma unroll
                    for (int j = 0; j < kTapsAhead; ++j) w1[i * kTapsAhead + j] = w[j];
                }
            } else if (ahead) {
#pragma unroll
                for (int i = 0; i < V; ++i)
#pragma unroll
                    for (int j = 0; j < kTapsAhead; ++j)
                        if ((uint32_t)j < p.taps) w1[i * kTapsAhead + j] = p.conv_w[((size_t)c + i) * p.taps + j];
            }
            find_window();
            if (ahead) {
#pragma unroll
                for (int j = 0; j + 1 < kTapsAhead; ++j)
                    if ((uint32_t)j + 1 < p.taps) win1[j] = ldc<V>(window + (size_t)j * d + c);
            }
            u1 = join_and_read<SM, V>(p, Mix<SM>(p), old, src, c);
#pragma unroll
            for (int i = 0; i < V; ++i) ss = fmaf(u1.v[i], u1.v[i], ss);
        }
    } else {
        find_window();
        const Mix<SM> m(p);
        for (uint32_t c = tid * V; c < d; c += NT * V) {
            const Cols<V> u = join_and_read<SM, V>(p, m, Copies<SM, V>(p, src, c), src, c);
            if (!p.h) continue;
            stc<V>(s_u + c, u);
#pragma unroll
            for (int i = 0; i < V; ++i) ss = fmaf(u.v[i], u.v[i], ss);
        }
    }
    if (!p.h) return; // (the same for every thread)
    ss = wave_sum(ss);
    if ((tid & 63) == 0) s_red[tid >> 6] = ss;
    __syncthreads();
    float total = 0.0f;
#pragma unroll
    for (int w = 0; w < NT / 64; ++w) total += s_red[w];
    const float inv = 1.0f / sqrtf(total / (float)d + p.eps);
    float* h = p.h + (size_t)r * d;
    for (uint32_t c = tid * V; c < d; c += NT * V) {
        const Cols<V> u = ONE ? u1 : ldc<V>(s_u + c), sc = ONE ? sc1 : ldc<V>(p.scales + c);
        Cols<V> own, acc;
#pragma unroll
        for (int i = 0; i < V; ++i) own.v[i] = u.v[i] * inv * (sc.v[i] + p.offset), acc.v[i] = 0.0f;
        if (!p.conv_w) {
            stc<V>(h + c, own);
            continue;
        }
        // taps in tap order, as causal_conv_rows adds them; the window moves on by this row
        auto tap = [&](uint32_t j, Cols<V> in, auto weight) {
            if (p.taps - 1 - j > t) {
#pragma unroll
                for (int i = 0; i < V; ++i) in.v[i] = 0.0f;
            }
#pragma unroll
            for (int i = 0; i < V; ++i) acc.v[i] = fmaf(weight(i), in.v[i], acc.v[i]);
            if (j) stc<V>(window + (size_t)(j - 1) * d + c, in);
        };
        float last[V];
        if (ahead) {
#pragma unroll
            for (int j = 0; j + 1 < kTapsAhead; ++j)
                if ((uint32_t)j + 1 < p.taps) tap(j, win1[j], [&](int i) { return w1[i * kTapsAhead + j]; });
#pragma unroll
            for (int i = 0; i < V; ++i)
#pragma unroll
                for (int j = 0; j < kTapsAhead; ++j)
                    if ((uint32_t)j + 1 == p.taps) last[i] = w1[i * kTapsAhead + j];
        } else {
            const float* w = p.conv_w + (size_t)c * p.taps;
            for (uint32_t j = 0; j + 1 < p.taps; ++j) tap(j, ldc<V>(window + (size_t)j * d + c), [&](int i) { return w[i * p.taps + j]; });
#pragma unroll
            for (int i = 0; i < V; ++i) last[i] = w[i * p.taps + p.taps - 1];
        }
        if (p.taps > 1) stc<V>(window + (size_t)(p.taps - 2) * d + c, own);
#pragma unroll
        for (int i = 0; i < V; ++i) acc.v[i] = own.v[i] + fmaf(last[i], own.v[i], acc.v[i]);
        stc<V>(h + c, acc);
    }
}

template <int SM, int V, int NT> uzu_status launch_as(hipStream_t s, const HyperStepParams& p) {
    if (p.d <= (uint32_t)NT * V) return launch_check([&] { hipLaunchKernelGGL((hyper_step_kernel<SM, V, NT, true>), dim3(p.rows), dim3(NT), 0, s, p); }, "hyper_step");
    static LdsLimit lim;
    const size_t lds = p.h ? (size_t)p.d * 4 : 0;
    raise_lds_limit(lim, (const void*)hyper_step_kernel<SM, V, NT, false>, lds);
    return launch_check([&] { hipLaunchKernelGGL((hyper_step_kernel<SM, V, NT, false>), dim3(p.rows), dim3(NT), lds, s, p); }, "hyper_step");
}
// few rows (one workgroup per row leaves the chip idle): wider workgroups
template <int SM> uzu_status launch(hipStream_t s, const HyperStepParams& p, bool vec) {
    if (!vec) return launch_as<SM, 1, 256>(s, p);
    return p.rows <= 64 ? launch_as<SM, 4, 512>(s, p) : launch_as<SM, 4, 256>(s, p);
}

} // namespace

uzu_status hyper_step(hipStream_t s, const HyperStepParams& p) {
    if (!p.rows) return UZU_OK;
    UZU_REQUIRE(p.src && p.streams && p.d && (!p.y || p.join) && (!p.h || p.scales) && (!p.dst || p.y), "hyper_step: null argument");
    UZU_UNSUPPORTED(p.streams > kHyperMaxStreams || p.d > kHyperMaxWidth, "hyper_step: %u streams of width %u (at most %u of %u)", p.streams, p.d, kHyperMaxStreams, kHyperMaxWidth);
    UZU_REQUIRE(!p.conv_w || (p.h && p.taps >= 1 && (p.taps == 1 || (p.states && p.spans && p.row_seq)) && !p.row_index), "hyper_step: an input convolution needs the pass's spans and windows");
    const uintptr_t at = (uintptr_t)p.src | (uintptr_t)p.dst | (uintptr_t)p.y | (uintptr_t)p.h | (uintptr_t)p.scales | (uintptr_t)p.sum_out | (uintptr_t)p.conv_w;
    const bool vec = p.d % 4 == 0 && p.src_stride % 4 == 0 && p.dst_stride % 4 == 0 && p.state_offset % 4 == 0 && at % 16 == 0;
    if (p.streams <= 2) return launch<2>(s, p, vec);
    if (p.streams <= 4) return launch<4>(s, p, vec);
    if (p.streams <= 8) return launch<8>(s, p, vec);
    return launch<16>(s, p, vec);
}

} // namespace k
} // namespace uzu
