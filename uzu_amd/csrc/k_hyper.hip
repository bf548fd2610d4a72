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

// a workgroup per row.  SM: most copies (p.streams <= SM); V: columns per thread and step (4 where rows are 16-byte aligned, else 1); SX: the copies are stored
template <int SM, int V>
__global__ void __launch_bounds__(256) hyper_step_kernel(HyperStepParams p) {
    extern __shared__ float s_u[]; // [d]: what the sublayer reads, in front of its norm (a thread reads back its own columns only)
    __shared__ float s_red[4];
    const uint32_t r = blockIdx.x, src = p.row_index ? p.row_index[r] : r, tid = threadIdx.x, d = p.d;
    const uint32_t S = p.streams;
    const float* x = p.src + (size_t)src * d;
    float* dst = p.dst ? p.dst + (size_t)src * d : nullptr;
    const float* y = p.y ? p.y + (size_t)src * d : nullptr;
    float w_in[SM], w_out[SM], w_mix[SM][SM];
#pragma unroll
    for (int a = 0; a < SM; ++a) {
        const bool on = (uint32_t)a < S;
        w_in[a] = on ? (p.read ? p.read[a] : 1.0f) : 0.0f;
        w_out[a] = on && y ? p.mult * p.join[S + a] : 0.0f;
#pragma unroll
        for (int b = 0; b < SM; ++b) w_mix[a][b] = on && (uint32_t)b < S && y ? p.join[2 * S + a * S + b] : 0.0f;
    }
    float ss = 0.0f;
    for (uint32_t c = tid * V; c < d; c += 256 * V) {
        Cols<V> old[SM], yv;
#pragma unroll
        for (int a = 0; a < SM; ++a)
            if ((uint32_t)a < S) old[a] = ldc<V>(x + a * p.src_stride + c);
        Cols<V> u, sum;
#pragma unroll
        for (int i = 0; i < V; ++i) u.v[i] = sum.v[i] = 0.0f;
        if (y) yv = ldc<V>(y + c);
#pragma unroll
        for (int b = 0; b < SM; ++b) {
            if ((uint32_t)b >= S) continue;
            Cols<V> now;
            if (y) {
#pragma unroll
                for (int i = 0; i < V; ++i) {
                    float v = 0.0f;
#pragma unroll
                    for (int a = 0; a < SM; ++a)
                        if ((uint32_t)a < S) v = fmaf(w_mix[a][b], old[a].v[i], v);
                    now.v[i] = fmaf(w_out[b], yv.v[i], v);
                }
                if (dst) stc<V>(dst + b * p.dst_stride + c, now);
            } else {
                now = old[b];
            }
#pragma unroll
            for (int i = 0; i < V; ++i) u.v[i] = fmaf(w_in[b], now.v[i], u.v[i]), sum.v[i] += now.v[i];
        }
        if (p.sum_out) stc<V>(p.sum_out + (size_t)src * d + c, sum);
        if (p.h) {
            stc<V>(s_u + c, u);
#pragma unroll
            for (int i = 0; i < V; ++i) ss = fmaf(u.v[i], u.v[i], ss);
        }
    }
    if (!p.h) return; // (the same for every thread)
    ss = wave_sum(ss);
    if ((tid & 63) == 0) s_red[tid >> 6] = ss;
    __syncthreads();
    const float inv = 1.0f / sqrtf((s_red[0] + s_red[1] + s_red[2] + s_red[3]) / (float)d + p.eps);
    float* h = p.h + (size_t)r * d;
    float* window = nullptr;
    bool first_rows = false; // the window's older entries stand in front of position 0
    uint32_t t = 0;
    if (p.conv_w && p.taps > 1) {
        const uint32_t z = p.row_seq[r];
        t = p.spans[z].start;
        window = p.states[z] + p.state_offset;
        first_rows = t < p.taps - 1;
    }
    for (uint32_t c = tid * V; c < d; c += 256 * V) {
        const Cols<V> u = ldc<V>(s_u + c), sc = ldc<V>(p.scales + c);
        Cols<V> own, acc;
#pragma unroll
        for (int i = 0; i < V; ++i) own.v[i] = u.v[i] * inv * (sc.v[i] + p.offset);
        if (!p.conv_w) {
            stc<V>(h + c, own);
            continue;
        }
        // the one row of its sequence: the convolution over the carried window (taps in tap order, as causal_conv_rows adds them), which moves on by this row
#pragma unroll
        for (int i = 0; i < V; ++i) acc.v[i] = 0.0f;
        const float* w = p.conv_w + (size_t)c * p.taps;
        for (uint32_t j = 0; j + 1 < p.taps; ++j) {
            Cols<V> in = ldc<V>(window + (size_t)j * d + c);
            if (first_rows && p.taps - 1 - j > t) {
#pragma unroll
                for (int i = 0; i < V; ++i) in.v[i] = 0.0f;
            }
#pragma unroll
            for (int i = 0; i < V; ++i) acc.v[i] = fmaf(w[i * p.taps + j], in.v[i], acc.v[i]);
            if (j) stc<V>(window + (size_t)(j - 1) * d + c, in);
        }
        if (p.taps > 1) stc<V>(window + (size_t)(p.taps - 2) * d + c, own);
#pragma unroll
        for (int i = 0; i < V; ++i) acc.v[i] = own.v[i] + fmaf(w[i * p.taps + p.taps - 1], own.v[i], acc.v[i]);
        stc<V>(h + c, acc);
    }
}

template <int SM> uzu_status launch(hipStream_t s, const HyperStepParams& p, bool vec) {
    const size_t lds = p.h ? (size_t)p.d * 4 : 0;
    if (vec) {
        static LdsLimit lim;
        raise_lds_limit(lim, (const void*)hyper_step_kernel<SM, 4>, lds);
        return launch_check([&] { hipLaunchKernelGGL((hyper_step_kernel<SM, 4>), dim3(p.rows), dim3(256), lds, s, p); }, "hyper_step");
    }
    static LdsLimit lim;
    raise_lds_limit(lim, (const void*)hyper_step_kernel<SM, 1>, lds);
    return launch_check([&] { hipLaunchKernelGGL((hyper_step_kernel<SM, 1>), dim3(p.rows), dim3(256), lds, s, p); }, "hyper_step");
}

} // namespace

uzu_status hyper_step(hipStream_t s, const HyperStepParams& p) {
    if (!p.rows) return UZU_OK;
    UZU_REQUIRE(p.src && p.streams && p.d && (!p.y || p.join) && (!p.h || p.scales) && (!p.dst || p.y), "hyper_step: null argument");
    UZU_UNSUPPORTED(p.streams > kHyperMaxStreams || p.d > kHyperMaxWidth, "hyper_step: %u streams of width %u (at most %u of %u)", p.streams, p.d, kHyperMaxStreams, kHyperMaxWidth);
    UZU_REQUIRE(!p.conv_w || (p.h && p.taps >= 1 && (p.taps == 1 || (p.states && p.spans && p.row_seq)) && !p.row_index), "hyper_step: an input convolution needs the pass's spans and windows");
    const uintptr_t at = (uintptr_t)p.src | (uintptr_t)p.dst | (uintptr_t)p.y | (uintptr_t)p.h | (uintptr_t)p.scales | (uintptr_t)p.sum_out;
    const bool vec = p.d % 4 == 0 && p.src_stride % 4 == 0 && p.dst_stride % 4 == 0 && p.state_offset % 4 == 0 && at % 16 == 0;
    if (p.streams <= 2) return launch<2>(s, p, vec);
    if (p.streams <= 4) return launch<4>(s, p, vec);
    if (p.streams <= 8) return launch<8>(s, p, vec);
    return launch<16>(s, p, vec);
}

} // namespace k
} // namespace uzu
