// k_window_attention.hip -- attention over a per-position cache of rotated keys and values for the f32-stream designs (kernels_stream32.h): rotation + key
// scaling + cache append, and the attention core with grouped heads, a soft cap on the scores, a causal sliding window and sink terms in the softmax denominator.
//
// Scores, softmax weights and the weighted sums are f32 whatever the cache holds (bf16 rows in the serving precision, f32 rows in the full-f32 mode).  A row's
// keys are walked in blocks of 64 counted from the first key the row sees, so the order of every sum depends on the row's position and the window only: not on
// how a prompt was cut into passes, and not on what else a pass carries.
#include "device_utils.h"
#include "kernels_stream32.h"

namespace uzu {
namespace k {

namespace {

__device__ __forceinline__ float cache_ld(const void* p, uint32_t is_bf16, size_t i) { return is_bf16 ? bf16_to_f32(((const uint16_t*)p)[i]) : ((const float*)p)[i]; }
__device__ __forceinline__ void cache_st(void* p, uint32_t is_bf16, size_t i, float v) {
    if (is_bf16) ((uint16_t*)p)[i] = f32_to_bf16(v);
    else ((float*)p)[i] = v;
}

// a workgroup per row (256 threads; few rows: 1024, so that the heads' norms run side by side): query pairs in place, key pairs (+ the unrotated tail) to the cache or in place, values to the cache
__global__ void __launch_bounds__(1024) rope_append_kernel(RopeAppendParams p) {
    const uint32_t r = blockIdx.x;
    const uint32_t z = p.row_seq[r];
    const SeqSpan sp = p.spans[z];
    const uint32_t t = sp.start + (r - sp.row0);
    float* row = p.qkv + (size_t)r * p.ld;
    const uint32_t half = p.rope_dim / 2;
    const float* cs = p.cosines + (size_t)t * p.rope_dim;
    const float* sn = p.sines + (size_t)t * p.rope_dim;
    // values first, as projected: with v_col == k_col the values are the keys in front of their norm and rotation
    if (p.kv_heads && p.value_caches) {
        void* vc = p.value_caches[z];
        const size_t vrow = (size_t)t * p.kv_heads * p.vdim;
        for (uint32_t idx = threadIdx.x; idx < p.kv_heads * p.vdim; idx += blockDim.x) cache_st(vc, p.cache_bf16, vrow + idx, row[p.v_col + idx]);
        __syncthreads();
    }
    if (p.norm_whole && (p.q_norm || p.k_norm)) { // one RMS norm over all query coordinates of the row, one over all key coordinates: 256 strided partial sums, a fixed tree
        __shared__ float s_red[256];
        for (int pass = 0; pass < 2; ++pass) {
            const float* w = pass ? p.k_norm : p.q_norm;
            const uint32_t n = pass ? p.kv_heads * p.dim : p.heads * p.dim;
            if (!w || !n) continue;
            float* h = pass ? row + p.k_col : row;
            float ss = 0.0f;
            for (uint32_t i = threadIdx.x; i < n; i += 256) ss = fmaf(h[i], h[i], ss);
            s_red[threadIdx.x] = ss;
            __syncthreads();
            for (uint32_t wd = 128; wd > 0; wd >>= 1) {
                if (threadIdx.x < wd) s_red[threadIdx.x] += s_red[threadIdx.x + wd];
                __syncthreads();
            }
            const float inv = 1.0f / sqrtf(s_red[0] / (float)n + p.norm_eps);
            __syncthreads();
            for (uint32_t i = threadIdx.x; i < n; i += 256) h[i] = h[i] * inv * w[i];
        }
        __syncthreads();
    } else if (p.q_norm || p.k_norm) { // a wave per head: x <- x / sqrt(mean(x^2) + eps) * w over the head's coordinates, in front of the rotation
        const uint32_t lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
        for (uint32_t a = wave; a < p.heads + p.kv_heads; a += blockDim.x >> 6) {
            const bool is_q = a < p.heads;
            const float* w = is_q ? p.q_norm : p.k_norm;
            if (!w) continue;
            float* h = is_q ? row + (size_t)a * p.dim : row + p.k_col + (size_t)(a - p.heads) * p.dim;
            float ss = 0.0f;
            for (uint32_t i = lane; i < p.dim; i += 64) ss = fmaf(h[i], h[i], ss);
            ss = wave_sum(ss);
            const float inv = 1.0f / sqrtf(ss / (float)p.dim + p.norm_eps);
            for (uint32_t i = lane; i < p.dim; i += 64) h[i] = h[i] * inv * w[i];
        }
        __syncthreads();
    }
    for (uint32_t idx = threadIdx.x; idx < p.heads * half; idx += blockDim.x) {
        const uint32_t a = idx / half, i = idx - a * half;
        float* h = row + (size_t)a * p.dim;
        const uint32_t iu = p.interleaved ? 2 * i : i, iv = p.interleaved ? 2 * i + 1 : i + half;
        const float u = h[iu], v = h[iv], c = cs[i], s = sn[i];
        h[iu] = u * c - v * s;
        h[iv] = v * c + u * s;
    }
    if (!p.kv_heads) return;
    const float ks = p.key_scale;
    void* kc = p.key_caches ? p.key_caches[z] : nullptr;
    const size_t krow = (size_t)t * p.kv_heads * p.dim;
    for (uint32_t idx = threadIdx.x; idx < p.kv_heads * p.dim; idx += blockDim.x) {
        const uint32_t g = idx / p.dim, c = idx - g * p.dim;
        float* h = row + p.k_col + (size_t)g * p.dim;
        if (c >= p.rope_dim) {
            const float a = h[c] * ks;
            if (kc) cache_st(kc, p.cache_bf16, krow + idx, a);
            else h[c] = a;
        } else if (p.interleaved ? (c & 1) == 0 : c < half) { // the thread of a pair's first coordinate turns the pair
            const uint32_t step = p.interleaved ? 1 : half, i = p.interleaved ? c >> 1 : c;
            const float u = h[c], v = h[c + step], co = cs[i], s = sn[i];
            const float a = (u * co - v * s) * ks, b = (v * co + u * s) * ks;
            if (kc) cache_st(kc, p.cache_bf16, krow + idx, a), cache_st(kc, p.cache_bf16, krow + idx + step, b);
            else h[c] = a, h[c + step] = b;
        }
    }
}
// The same behind a causal convolution of the row, for passes of one row per sequence: a workgroup takes whole query heads, whole key heads, or 256 of the channels behind
// them (values to the cache, what stands behind the values back to the rows).  A channel's window is replaced by the thread that alone reads it; taps in tap order, as in
// causal_conv_rows.
__device__ __forceinline__ uint32_t conv_rope_heads_per_block(uint32_t dim) { return dim < 256 ? 256 / dim : 1; }
template <int T> __device__ __forceinline__ float conv_channel(const CausalConvParams& c, const SeqSpan& sp, float* window, uint32_t r, uint32_t ch) {
    float in[T], w[T];
    in[T - 1] = c.x[(size_t)r * c.ldx + c.x_col + ch];
    float acc = c.bias ? c.bias[ch] : 0.0f;
#pragma unroll
    for (int j = 0; j < T; ++j) {
        w[j] = c.w[(size_t)ch * T + j];
        if (j < T - 1) in[j] = (uint32_t)(T - 1 - j) <= sp.start ? window[(size_t)j * c.channels + ch] : 0.0f; // (in front of position 0: zeros)
    }
#pragma unroll
    for (int j = 0; j < T; ++j) acc = fmaf(w[j], in[j], acc);
    if (c.act == 1 && ch >= c.act_from) acc = acc / (1.0f + expf(-acc));
    if (c.add_input) acc = in[T - 1] + acc;
#pragma unroll
    for (int j = 0; j < T - 1; ++j) window[(size_t)j * c.channels + ch] = in[j + 1];
    return acc;
}
template <int T> __global__ void __launch_bounds__(256) conv_rope_append_kernel(RopeAppendParams p, CausalConvParams c) {
    extern __shared__ float s_h[]; // the block's heads
    const uint32_t r = blockIdx.x, z = p.row_seq[r], hpb = conv_rope_heads_per_block(p.dim), qb = (p.heads + hpb - 1) / hpb, kb = (p.kv_heads + hpb - 1) / hpb;
    const SeqSpan sp = p.spans[z];
    const uint32_t t = sp.start;
    float* window = c.states[z] + c.state_offset;
    float* row = p.qkv + (size_t)r * p.ld;
    if (blockIdx.y >= qb + kb) { // values and what stands behind them
        const uint32_t ch = p.v_col + (blockIdx.y - qb - kb) * 256 + threadIdx.x;
        if (ch >= c.channels) return;
        const float v = conv_channel<T>(c, sp, window, r, ch);
        if (ch < p.v_col + p.kv_heads * p.vdim) cache_st(p.value_caches[z], p.cache_bf16, (size_t)t * p.kv_heads * p.vdim + (ch - p.v_col), v);
        else row[ch] = v;
        return;
    }
    const bool is_q = blockIdx.y < qb;
    const uint32_t h0 = (is_q ? blockIdx.y : blockIdx.y - qb) * hpb, heads = is_q ? p.heads : p.kv_heads, n = (h0 + hpb < heads ? hpb : heads - h0) * p.dim;
    const uint32_t c0 = (is_q ? 0 : p.k_col) + h0 * p.dim, half = p.rope_dim / 2;
    for (uint32_t i = threadIdx.x; i < n; i += 256) s_h[i] = conv_channel<T>(c, sp, window, r, c0 + i);
    __syncthreads();
    const float *cs = p.cosines + (size_t)t * p.rope_dim, *sn = p.sines + (size_t)t * p.rope_dim;
    void* kc = is_q ? nullptr : p.key_caches[z];
    const float scale = is_q ? 1.0f : p.key_scale;
    for (uint32_t i = threadIdx.x; i < n; i += 256) {
        const uint32_t d = i % p.dim, head = i - d;
        float v = s_h[i];
        if (d < p.rope_dim) {
            const uint32_t pair = p.interleaved ? d >> 1 : d < half ? d : d - half;
            const bool first = p.interleaved ? (d & 1) == 0 : d < half;
            const uint32_t iu = head + (p.interleaved ? 2 * pair : pair), iv = iu + (p.interleaved ? 1 : half);
            const float a = s_h[iu], b = s_h[iv], co = cs[pair], si = sn[pair];
            v = first ? a * co - b * si : b * co + a * si;
        }
        v *= scale;
        if (is_q) row[c0 + i] = v;
        else cache_st(kc, p.cache_bf16, (size_t)t * p.kv_heads * p.dim + h0 * p.dim + i, v);
    }
}

// ---- the simple form: a wave per (row, head).  Keys in blocks of 64 from the row's first visible key: a lane scores one key of the block (the whole dot
// product, the query staged in LDS), the block's weights go through LDS, then a lane owns value coordinates lane, lane + 64, ... of the running sum.
constexpr uint32_t kMaxVecPerLane = 8; // value widths up to 512
__global__ void __launch_bounds__(64) window_attention_simple_kernel(WindowAttentionParams p) {
    extern __shared__ float s_mem[]; // [dim] query + [64] weights
    float* s_q = s_mem;
    float* s_p = s_mem + p.dim;
    const uint32_t r = blockIdx.x, a = blockIdx.y, lane = threadIdx.x;
    const uint32_t z = p.row_seq[r];
    const SeqSpan sp = p.spans[z];
    const uint32_t t = sp.start + (r - sp.row0);
    const uint32_t g = a / (p.heads / p.kv_heads);
    const void* K = p.key_caches[z];
    const void* V = p.value_caches[z];
    uint32_t lo = (p.window && t + 1 > p.window) ? t + 1 - p.window : 0u;
    if (p.chunk) lo = max(lo, t / p.chunk * p.chunk);
    const float hscale = p.head_scale ? p.scale * p.head_scale[a] : p.scale;
    const float* q = p.q + (size_t)r * p.ldq + (size_t)a * p.dim;
    for (uint32_t c = lane; c < p.dim; c += 64) s_q[c] = q[c];
    __syncthreads();
    float m = p.sinks ? p.sinks[a] : -INFINITY, l = p.sinks ? 1.0f : 0.0f;
    float acc[kMaxVecPerLane];
#pragma unroll
    for (uint32_t i = 0; i < kMaxVecPerLane; ++i) acc[i] = 0.0f;
    const size_t kpitch = (size_t)p.kv_heads * p.dim, vpitch = (size_t)p.kv_heads * p.vdim;
    for (uint32_t j0 = lo; j0 <= t; j0 += 64) {
        const uint32_t j = j0 + lane;
        float s = -INFINITY;
        if (j <= t) {
            const size_t base = (size_t)j * kpitch + (size_t)g * p.dim;
            float dot = 0.0f;
            if (p.cache_bf16) {
                const uint16_t* kr = (const uint16_t*)K + base;
                if ((p.dim & 7) == 0 && (((uintptr_t)kr) & 15) == 0) {
                    for (uint32_t c = 0; c < p.dim; c += 8) {
                        const uint4 kv = *(const uint4*)(kr + c);
                        const uint32_t w[4] = {kv.x, kv.y, kv.z, kv.w};
#pragma unroll
                        for (int i = 0; i < 4; ++i) {
                            dot = fmaf(s_q[c + 2 * i], bits_to_f32(w[i] << 16), dot);
                            dot = fmaf(s_q[c + 2 * i + 1], bits_to_f32(w[i] & 0xFFFF0000u), dot);
                        }
                    }
                } else {
                    for (uint32_t c = 0; c < p.dim; ++c) dot = fmaf(s_q[c], bf16_to_f32(kr[c]), dot);
                }
            } else {
                const float* kr = (const float*)K + base;
                for (uint32_t c = 0; c < p.dim; ++c) dot = fmaf(s_q[c], kr[c], dot);
            }
            s = dot * hscale;
            if (p.soft_cap != 0.0f) s = p.soft_cap * tanhf(s / p.soft_cap);
            if (p.dist_bias) s += p.dist_bias[(size_t)min(t - j, p.dist_rows - 1) * p.heads + a];
        }
        const float m_new = fmaxf(m, wave_max(s));
        const float w = j <= t ? expf(s - m_new) : 0.0f;
        const float corr = expf(m - m_new); // (first block without a sink: exp(-inf) = 0 against l = 0 and zero sums)
        l = l * corr + wave_sum(w);
        m = m_new;
        __syncthreads();
        s_p[lane] = w;
        __syncthreads();
        const uint32_t nk = t - j0 + 1 < 64 ? t - j0 + 1 : 64;
#pragma unroll
        for (uint32_t i = 0; i < kMaxVecPerLane; ++i) {
            const uint32_t c = lane + 64 * i;
            if (c >= p.vdim) break;
            float sum = acc[i] * corr;
            const size_t vb = (size_t)j0 * vpitch + (size_t)g * p.vdim + c;
            for (uint32_t jj = 0; jj < nk; ++jj) sum = fmaf(s_p[jj], cache_ld(V, p.cache_bf16, vb + (size_t)jj * vpitch), sum);
            acc[i] = sum;
        }
    }
    float* o = p.out + (size_t)r * p.ldo + (size_t)a * p.vdim;
    const float og = p.gate ? p.out_scale / (1.0f + expf(-p.gate[(size_t)r * p.ldgate + a])) : p.out_scale;
#pragma unroll
    for (uint32_t i = 0; i < kMaxVecPerLane; ++i) {
        const uint32_t c = lane + 64 * i;
        if (c >= p.vdim) break;
        o[c] = acc[i] / l * og; // (og = 1: the value itself)
    }
}

} // namespace

uzu_status rope_append(hipStream_t s, const RopeAppendParams& p) {
    if (!p.rows) return UZU_OK;
    UZU_REQUIRE(p.qkv && p.spans && p.row_seq && p.heads && p.dim, "rope_append: null argument");
    UZU_REQUIRE(p.rope_dim % 2 == 0 && p.rope_dim <= p.dim && (!p.rope_dim || (p.cosines && p.sines)), "rope_append: rotation width %u of a head of %u (even, with its tables)", p.rope_dim, p.dim);
    UZU_REQUIRE(!p.kv_heads || ((p.key_caches != nullptr) == (p.value_caches != nullptr)), "rope_append: key and value caches come together");
    UZU_REQUIRE(p.v_col != p.k_col || !p.kv_heads || (p.vdim == p.dim && p.value_caches), "rope_append: values that are the key rows have the keys' width and go to a cache");
    return launch_check([&] { hipLaunchKernelGGL(rope_append_kernel, dim3(p.rows), dim3(p.rows <= 64 && !p.norm_whole ? 1024 : 256), 0, s, p); }, "rope_append");
}

bool conv_rope_append_supported(const RopeAppendParams& p, const CausalConvParams& c) {
    return c.max_count == 1 && c.taps >= 1 && c.taps <= 4 && !p.q_norm && !p.k_norm && p.kv_heads && p.v_col != p.k_col && p.key_caches && p.value_caches && p.dim <= 8192;
}

uzu_status conv_rope_append(hipStream_t s, const RopeAppendParams& p, const CausalConvParams& c) {
    if (!p.rows) return UZU_OK;
    UZU_REQUIRE(conv_rope_append_supported(p, c) && c.x && c.w && (c.states || c.taps == 1) && c.out == p.qkv && c.ldo == p.ld && !c.o_col && c.rows == p.rows && c.x != c.out,
                "conv_rope_append: one row per sequence, 1 .. 4 taps, no head norms, the convolution's result in place of the packed rows");
    UZU_REQUIRE(p.spans && p.row_seq && p.heads && p.dim && p.rope_dim % 2 == 0 && p.rope_dim <= p.dim && (!p.rope_dim || (p.cosines && p.sines)), "conv_rope_append: an even rotation width with its tables");
    UZU_REQUIRE(p.k_col == p.heads * p.dim && p.v_col == p.k_col + p.kv_heads * p.dim && p.v_col + p.kv_heads * p.vdim <= c.channels && c.x_col + c.channels <= c.ldx && c.channels <= c.ldo,
                "conv_rope_append: rows of queries | keys | values (| ..)");
    const uint32_t hpb = p.dim < 256 ? 256 / p.dim : 1, blocks = (p.heads + hpb - 1) / hpb + (p.kv_heads + hpb - 1) / hpb + (c.channels - p.v_col + 255) / 256;
    UZU_REQUIRE(blocks <= 65535, "conv_rope_append: too many channels for one launch");
#define UZU_CR(T) case T: return launch_check([&] { hipLaunchKernelGGL(conv_rope_append_kernel<T>, dim3(p.rows, blocks), dim3(256), (size_t)hpb * p.dim * 4, s, p, c); }, "conv_rope_append")
    switch (c.taps) {
        UZU_CR(1);
        UZU_CR(2);
        UZU_CR(3);
        UZU_CR(4);
        default: return UZU_ERR_INVALID_ARGUMENT;
    }
#undef UZU_CR
}

uzu_status window_attention_mfma(hipStream_t s, const WindowAttentionParams& p); // k_window_attention_mfma.hip

uzu_status window_attention(hipStream_t s, const WindowAttentionParams& params) {
    WindowAttentionParams p = params;
    if (!p.rows) return UZU_OK;
    if (!p.ldo) p.ldo = p.heads * p.vdim;
    if (p.out_scale == 0.0f) p.out_scale = 1.0f;
    UZU_REQUIRE(p.ldo >= p.heads * p.vdim, "window_attention: result rows of pitch %u", p.ldo);
    UZU_REQUIRE(p.q && p.out && p.key_caches && p.value_caches && p.spans && p.row_seq, "window_attention: null argument");
    UZU_REQUIRE(p.heads && p.kv_heads && p.heads % p.kv_heads == 0 && p.dim && p.vdim, "window_attention: %u query heads on %u key / value heads", p.heads, p.kv_heads);
    UZU_UNSUPPORTED(p.vdim > 64 * kMaxVecPerLane || p.dim > 8192, "window_attention: value width %u (at most %u)", p.vdim, 64 * kMaxVecPerLane);
    UZU_REQUIRE(!p.dist_bias || p.dist_rows, "window_attention: a distance bias without its rows");
    if (p.form == 2 || (p.form == 0 && window_attention_mfma_supported(p))) {
        UZU_UNSUPPORTED(!window_attention_mfma_supported(p), "window_attention: the matrix-core form does not take this shape");
        return window_attention_mfma(s, p);
    }
    UZU_REQUIRE(p.heads <= 65535, "window_attention: too many heads for one launch");
    return launch_check([&] { hipLaunchKernelGGL(window_attention_simple_kernel, dim3(p.rows, p.heads), dim3(64), (size_t)(p.dim + 64) * 4, s, p); }, "window_attention");
}

} // namespace k
} // namespace uzu
