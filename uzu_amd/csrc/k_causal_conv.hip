// k_causal_conv.hip -- a causal convolution over positions on every channel of a block of f32 rows, for the f32-stream designs (kernels_stream32.h): the input
// convolution of a sublayer (what the sublayer reads is h + conv(h)) and the short convolution with silu in front of a delta rule.
//
// Row r sits at position t of its sequence; tap j weighs the input of position t - (taps - 1) + j, so the last tap weighs the row itself.  Inputs in front of the
// pass come from the sequence's state (the last taps - 1 inputs, oldest first), inputs in front of position 0 are zeros whatever the state holds.  The taps are
// added in tap order whatever their source, so a row's result does not depend on how a prompt was cut into passes or on what else a pass carries.  The state is
// replaced by a launch of its own (thread = (sequence, channel)): the rows of the first launch read the old one.
#include "device_utils.h"
#include "kernels_stream32.h"

namespace uzu {
namespace k {

namespace {

// the inputs of positions end - (taps - 1) .. end - 1 of sequence z, channel c: from this pass's rows, the old window, or (in front of position 0) zeros
__device__ __forceinline__ void window_update(const CausalConvParams& p, const SeqSpan& sp, uint32_t z, uint32_t c) {
    float* cs = p.states[z] + p.state_offset;
    const uint32_t keep = p.taps - 1;
    for (uint32_t s = 0; s < keep; ++s) { // ascending: an old entry is read at index s + count > s before that index is written
        float v = 0.0f;
        if (s + sp.count >= keep) v = p.x[(size_t)(sp.row0 + (s + sp.count - keep)) * p.ldx + p.x_col + c];
        else if (sp.start + sp.count + s >= keep) v = cs[(size_t)(s + sp.count) * p.channels + c];
        cs[(size_t)s * p.channels + c] = v;
    }
}

// thread = (row, channel).  A sequence that brings ONE row (a decode step) has its window replaced here: the row's own thread is the only reader of the old one.
__global__ void __launch_bounds__(256) causal_conv_rows_kernel(CausalConvParams p) {
    const uint32_t r = blockIdx.x, c = blockIdx.y * 256 + threadIdx.x;
    if (c >= p.channels) return;
    const uint32_t z = p.row_seq[r];
    const SeqSpan sp = p.spans[z];
    const uint32_t i = r - sp.row0, t = sp.start + i;
    const float* state = p.taps > 1 ? p.states[z] + p.state_offset : nullptr;
    const float own = p.x[(size_t)r * p.ldx + p.x_col + c];
    float acc = p.bias ? p.bias[c] : 0.0f;
    for (uint32_t j = 0; j < p.taps; ++j) {
        const uint32_t back = p.taps - 1 - j;
        float xin = 0.0f;
        if (back == 0) xin = own;
        else if (back <= i) xin = p.x[(size_t)(r - back) * p.ldx + p.x_col + c];
        else if (back <= t) xin = state[(size_t)(p.taps - 1 - (back - i)) * p.channels + c]; // in front of the pass: the state's rows are positions start - (taps - 1) .. start - 1
        acc = fmaf(p.w[(size_t)c * p.taps + j], xin, acc);
    }
    if (p.act == 1 && c >= p.act_from) acc = acc / (1.0f + expf(-acc));
    if (p.add_input) acc = own + acc;
    p.out[(size_t)r * p.ldo + p.o_col + c] = acc;
    if (sp.count == 1 && p.taps > 1) window_update(p, sp, z, c);
}

// The same sums for many rows: thread = (four channels, kConvRows consecutive rows of the pass).  A channel's taps are loaded once, the last T - 1 input rows travel in
// registers; a row in front of which its sequence has fewer rows in this pass takes the older inputs from the state (or zeros), as above.
constexpr uint32_t kConvRows = 8;
template <int T>
__global__ void __launch_bounds__(256) causal_conv_block_kernel(CausalConvParams p) {
    const uint32_t c = (blockIdx.x * 256 + threadIdx.x) * 4, r0 = blockIdx.y * kConvRows;
    if (c >= p.channels) return;
    const uint32_t r1 = r0 + kConvRows < p.rows ? r0 + kConvRows : p.rows;
    const float* x = p.x + p.x_col + c;
    float w[4][T];
    f32x4_v past[T]; // past[b]: the input b rows back (past[0]: the row itself)
#pragma unroll
    for (int i = 0; i < 4; ++i)
#pragma unroll
        for (int j = 0; j < T; ++j) w[i][j] = p.w[((size_t)c + i) * T + j];
    const f32x4_v zero{0.f, 0.f, 0.f, 0.f}, bias = p.bias ? f32x4_v{p.bias[c], p.bias[c + 1], p.bias[c + 2], p.bias[c + 3]} : zero;
#pragma unroll
    for (int b = 0; b < T; ++b) past[b] = b && r0 >= (uint32_t)b ? *(const f32x4_v*)(x + (size_t)(r0 - b) * p.ldx) : zero;
#pragma unroll
    for (uint32_t k = 0; k < kConvRows; ++k) {
        const uint32_t r = r0 + k;
        if (r >= r1) break;
        past[0] = *(const f32x4_v*)(x + (size_t)r * p.ldx);
        const uint32_t z = p.row_seq[r];
        const SeqSpan sp = p.spans[z];
        const uint32_t i = r - sp.row0, t = sp.start + i;
        f32x4_v acc = bias;
#pragma unroll
        for (int j = 0; j < T; ++j) {
            const uint32_t back = T - 1 - j;
            f32x4_v in = past[back];
            if (back > i) in = back <= t ? *(const f32x4_v*)(p.states[z] + p.state_offset + (size_t)(T - 1 - (back - i)) * p.channels + c) : zero;
#pragma unroll
            for (int q = 0; q < 4; ++q) acc[q] = fmaf(w[q][j], in[q], acc[q]);
        }
#pragma unroll
        for (int q = 0; q < 4; ++q) {
            if (p.act == 1 && c + q >= p.act_from) acc[q] = acc[q] / (1.0f + expf(-acc[q]));
            if (p.add_input) acc[q] = past[0][q] + acc[q];
        }
        *(f32x4_v*)(p.out + (size_t)r * p.ldo + p.o_col + c) = acc;
        if (sp.count == 1 && T > 1)
            for (uint32_t q = 0; q < 4; ++q) window_update(p, sp, z, c + q);
#pragma unroll
        for (int b = T - 1; b > 0; --b) past[b] = past[b - 1];
    }
}

// thread = (sequence, channel): the windows of the sequences that bring several rows (their first rows' threads read the old window in the launch before)
__global__ void __launch_bounds__(256) causal_conv_commit_kernel(CausalConvParams p) {
    const uint32_t z = blockIdx.x, c = blockIdx.y * 256 + threadIdx.x;
    if (c >= p.channels) return;
    const SeqSpan sp = p.spans[z];
    if (sp.count == 1) return; // done by the row's own thread
    window_update(p, sp, z, c);
}

// a wave per (row, head): x / sqrt(mean(x^2) + eps) * weight * gate
__global__ void __launch_bounds__(256) head_norm_gate_kernel(HeadNormGateParams p) {
    const uint32_t lane = threadIdx.x & 63, item = blockIdx.x * 4 + (threadIdx.x >> 6);
    if (item >= p.rows * p.heads) return;
    const uint32_t r = item / p.heads, a = item - r * p.heads;
    float* x = p.x + (size_t)r * p.ldx + (size_t)a * p.width;
    float ss = 0.0f;
    for (uint32_t i = lane; i < p.width; i += 64) ss = fmaf(x[i], x[i], ss);
    ss = wave_sum(ss);
    const float inv = 1.0f / sqrtf(ss / (float)p.width + p.eps);
    const float* g = p.gate ? p.gate + (size_t)r * p.ldgate + (size_t)a * p.width : nullptr;
    for (uint32_t i = lane; i < p.width; i += 64) {
        float v = x[i] * inv;
        if (p.weight) v *= p.weight[i];
        if (g) v *= p.gate_sigmoid ? 1.0f / (1.0f + expf(-g[i])) : g[i] / (1.0f + expf(-g[i]));
        x[i] = v;
    }
}

// a workgroup per (row, part): the first kGatedKeep coordinates travel in registers, their weights too (every load in front of the sum of squares), wider parts go over
// the rest in further steps
constexpr uint32_t kGatedUnroll = 4, kGatedKeep = 256 * kGatedUnroll;
__global__ void __launch_bounds__(256) gated_norm_rows_kernel(GatedNormParams p) {
    __shared__ float s_red[16];
    const uint32_t r = blockIdx.x, w = p.width / p.parts, c0 = blockIdx.y * w, tid = threadIdx.x;
    const float *y = p.y + (size_t)r * p.ldy + c0, *g = p.gate + (size_t)r * p.ldgate + c0, *wt = p.weight + c0;
    float* out = p.out + (size_t)r * p.ldo + c0;
    auto gated = [](float v, float z) { return v * (z / (1.0f + expf(-z))); };
    float yv[kGatedUnroll], gv[kGatedUnroll], wv[kGatedUnroll], ss = 0.0f;
#pragma unroll
    for (uint32_t u = 0; u < kGatedUnroll; ++u) {
        const uint32_t i = tid + u * 256;
        yv[u] = i < w ? y[i] : 0.0f, gv[u] = i < w ? g[i] : 0.0f, wv[u] = i < w ? wt[i] : 0.0f;
    }
#pragma unroll
    for (uint32_t u = 0; u < kGatedUnroll; ++u) {
        yv[u] = gated(yv[u], gv[u]);
        ss = fmaf(yv[u], yv[u], ss);
    }
    for (uint32_t i = tid + kGatedKeep; i < w; i += 256) {
        const float v = gated(y[i], g[i]);
        ss = fmaf(v, v, ss);
    }
    const float inv = p.out_scale / sqrtf(block_sum(ss, s_red) / (float)w + p.eps);
#pragma unroll
    for (uint32_t u = 0; u < kGatedUnroll; ++u) {
        const uint32_t i = tid + u * 256;
        if (i < w) out[i] = yv[u] * inv * wv[u];
    }
    for (uint32_t i = tid + kGatedKeep; i < w; i += 256) out[i] = gated(y[i], g[i]) * inv * wt[i]; // (out may be y: a thread replaces what it alone reads)
}

} // namespace

uzu_status gated_norm_rows(hipStream_t s, const GatedNormParams& p) {
    if (!p.rows) return UZU_OK;
    UZU_REQUIRE(p.y && p.gate && p.weight && p.out && p.width && p.parts && p.parts <= 65535 && p.width % p.parts == 0, "gated_norm: %u coordinates in %u equal parts", p.width, p.parts);
    return launch_check([&] { hipLaunchKernelGGL(gated_norm_rows_kernel, dim3(p.rows, p.parts), dim3(256), 0, s, p); }, "gated_norm_rows");
}

uzu_status causal_conv_rows(hipStream_t s, const CausalConvParams& p) {
    if (!p.rows) return UZU_OK;
    UZU_REQUIRE(p.x && p.out && p.w && (p.states || p.taps == 1) && p.spans && p.row_seq && p.channels && p.taps >= 1, "causal_conv: null argument");
    UZU_REQUIRE(p.x_col + p.channels <= p.ldx && p.o_col + p.channels <= p.ldo, "causal_conv: %u channels at columns %u / %u of rows of %u / %u", p.channels, p.x_col, p.o_col, p.ldx, p.ldo);
    UZU_REQUIRE(p.out != p.x || p.taps == 1, "causal_conv: a row reads earlier rows of the pass: the result goes to another block of rows");
    const uintptr_t at = (uintptr_t)(p.x + p.x_col) | (uintptr_t)(p.out + p.o_col);
    if (p.rows >= 64 && p.taps <= 6 && p.channels % 4 == 0 && p.ldx % 4 == 0 && p.ldo % 4 == 0 && p.state_offset % 4 == 0 && at % 16 == 0) {
        const dim3 grid((p.channels / 4 + 255) / 256, (p.rows + kConvRows - 1) / kConvRows);
        UZU_REQUIRE(grid.y <= 65535, "causal_conv: too many rows for one launch");
#define UZU_CONV(T) case T: return launch_check([&] { hipLaunchKernelGGL(causal_conv_block_kernel<T>, grid, dim3(256), 0, s, p); }, "causal_conv_block")
        switch (p.taps) {
            UZU_CONV(1);
            UZU_CONV(2);
            UZU_CONV(3);
            UZU_CONV(4);
            UZU_CONV(5);
            UZU_CONV(6);
        }
#undef UZU_CONV
    }
    return launch_check([&] { hipLaunchKernelGGL(causal_conv_rows_kernel, dim3(p.rows, (p.channels + 255) / 256), dim3(256), 0, s, p); }, "causal_conv_rows");
}

uzu_status causal_conv_commit(hipStream_t s, const CausalConvParams& p) {
    if (!p.rows || p.taps < 2 || p.max_count == 1) return UZU_OK; // (every sequence brings one row: the rows' launch has replaced the windows)
    UZU_REQUIRE(p.x && p.states && p.spans && p.nseq && p.channels, "causal_conv: null argument");
    return launch_check([&] { hipLaunchKernelGGL(causal_conv_commit_kernel, dim3(p.nseq, (p.channels + 255) / 256), dim3(256), 0, s, p); }, "causal_conv_commit");
}

uzu_status head_norm_gate_rows(hipStream_t s, const HeadNormGateParams& p) {
    if (!p.rows) return UZU_OK;
    UZU_REQUIRE(p.x && p.heads && p.width && p.heads * p.width <= p.ldx, "head_norm_gate: null argument");
    return launch_check([&] { hipLaunchKernelGGL(head_norm_gate_kernel, dim3((p.rows * p.heads + 3) / 4), dim3(256), 0, s, p); }, "head_norm_gate_rows");
}

} // namespace k
} // namespace uzu
