// k_decayed_state.hip -- linear attention over a decayed outer-product state whose decays come from the data, for the f32-stream designs
// (kernels_stream32.h::decayed_state): gated linear attention (a decay per head and key channel) and state-space duality (one decay per head and step).
//
// Per head a (reading query / key group a / (heads / groups)), with S [dim][vdim] the head's state and e_t the step's log decays (<= 0; a vector over the key
// channels, or one number):
//     S <- diag(e^(e_t)) S + k_t v_t^T,    o_t = q_t^T S (+ skip_a v_t)
// Everything is f32, products on the matrix cores included (f32 operands).  Decode-sized passes go token by token with the state in registers; prompts go in
// chunks of 64 rows, cut into four blocks of 16.  Decays over a stretch of rows are always exponentials of a SUM of that stretch's own log decays (never of a
// difference of running sums, and never a growing factor against a shrinking one), so neither a fast decay nor a long prompt costs accuracy or range:
//   row j of block J seen from row i of block I > J:  e^(suffix of j in J) * (whole blocks in between) * e^(prefix of i in I);  inside a block: running products.
#include <algorithm>

#include "device_utils.h"
#include "kernels_stream32.h"

namespace uzu {
namespace k {

namespace {

__device__ __forceinline__ float log_sigmoid_f32(float z) { return fminf(z, 0.0f) - log1pf(expf(-fabsf(z))); }
__device__ __forceinline__ float softplus_f32(float z) { return fmaxf(z, 0.0f) + log1pf(expf(-fabsf(z))); }

// one decay per head: the step size of a row (it multiplies the key) and the row's log decay
__device__ __forceinline__ float head_step(const DecayedStateParams& p, uint32_t r, uint32_t a) { return softplus_f32(p.decay[(size_t)r * p.lddecay + a] + p.dt_bias[a]); }
// a decay per key channel
__device__ __forceinline__ float channel_log_decay(const DecayedStateParams& p, uint32_t r, uint32_t a, uint32_t c) {
    return log_sigmoid_f32(p.decay[(size_t)r * p.lddecay + (size_t)a * p.dim + c]) * p.inv_temperature;
}

// ---- token by token.  grid (sequence * heads, ceil(vdim / 16)); thread = (column tid % 16, part tid / 16 of the key channels): it owns S[i][column] for
// i = part, part + 16, ...; a token's partial sums meet by lane exchange and then over the four waves in LDS, in a fixed order
template <int N, bool CHANNEL> // N: channels per thread (dim <= 16 N)
__global__ void __launch_bounds__(256) decayed_state_steps_kernel(DecayedStateParams p) {
    __shared__ float s_q[16 * N], s_k[16 * N], s_e[CHANNEL ? 16 * N : 1], s_v[16], s_red[4][16];
    const uint32_t z = blockIdx.x / p.heads, a = blockIdx.x % p.heads, g = a / (p.heads / p.groups);
    const uint32_t tid = threadIdx.x, cl = tid & 15, part = tid >> 4, wave = tid >> 6, col = blockIdx.y * 16 + cl;
    const SeqSpan sp = p.spans[z];
    if (!sp.count) return;
    const bool live = col < p.vdim;
    float* state = p.states[z] + (size_t)a * p.dim * p.vdim;
    float S[N];
#pragma unroll
    for (int n = 0; n < N; ++n) {
        const uint32_t i = part + 16 * n;
        S[n] = (sp.start && live && i < p.dim) ? state[(size_t)i * p.vdim + col] : 0.0f;
    }
    const float rate = CHANNEL ? 0.0f : expf(p.a_log[a]);
    for (uint32_t t = 0; t < sp.count; ++t) {
        const uint32_t r = sp.row0 + t;
        const float* row = p.rows_in + (size_t)r * p.ld;
        float decay = 0.0f, step = 1.0f;
        if (!CHANNEL) step = head_step(p, r, a), decay = expf(-rate * step);
        for (uint32_t c = tid; c < 16 * N; c += 256) { // (channels beyond dim: zeros, so that the padding rows of S stay zero)
            const bool in = c < p.dim;
            s_q[c] = in ? row[p.q_col + (size_t)g * p.dim + c] * p.q_scale : 0.0f;
            s_k[c] = in ? row[p.k_col + (size_t)g * p.dim + c] * step : 0.0f;
            if (CHANNEL) s_e[c] = in ? expf(channel_log_decay(p, r, a, c)) : 0.0f;
        }
        if (tid < 16) s_v[tid] = live ? row[p.v_col + (size_t)a * p.vdim + col] : 0.0f;
        __syncthreads();
        const float v = s_v[cl];
        float sum = 0.0f;
#pragma unroll
        for (int n = 0; n < N; ++n) {
            const uint32_t i = part + 16 * n;
            S[n] = fmaf(CHANNEL ? s_e[i] : decay, S[n], s_k[i] * v);
            sum = fmaf(S[n], s_q[i], sum);
        }
        sum += __shfl_xor(sum, 16, 64);
        sum += __shfl_xor(sum, 32, 64);
        if ((tid & 63) < 16) s_red[wave][cl] = sum;
        __syncthreads();
        if (tid < 16 && live) {
            float o = (s_red[0][cl] + s_red[1][cl]) + (s_red[2][cl] + s_red[3][cl]);
            if (p.skip) o = fmaf(p.skip[a], v, o);
            p.out[((size_t)r * p.heads + a) * p.vdim + col] = o;
        }
    }
    if (!live) return;
#pragma unroll
    for (int n = 0; n < N; ++n) {
        const uint32_t i = part + 16 * n;
        if (i < p.dim) state[(size_t)i * p.vdim + col] = S[n];
    }
}

// ---- in chunks of 64 rows:
//   local      A_c = sum_j diag(decay of the rows behind j) k_j v_j^T,  D_c = the chunk's whole decay                       (parallel over chunks)
//   scan       S_(c+1) = diag(D_c) S_c + A_c, the sequence's state in front and behind                                     (chunk after chunk, element-wise)
//   out        o_i = (decayed q_i)^T S_c + sum_(j <= i) <q_i, decay(j -> i) k_j> v_j                                        (parallel over chunks)
// ws holds per (chunk of the pass, head) [dim][vdim] -- first A_c, then S_c in its place -- and behind all of them D_c ([dim], one decay per head: [1]).
constexpr uint32_t kChunk = 64, kBlock = 16;
typedef float f32x16_m __attribute__((ext_vector_type(16)));
typedef float f32x4_m __attribute__((ext_vector_type(4)));

__device__ __forceinline__ bool find_chunk(const DecayedStateParams& p, uint32_t index, uint32_t& z, uint32_t& c, SeqSpan& sp) {
    for (z = 0; z < p.nseq; ++z) {
        sp = p.spans[z];
        const uint32_t n = (sp.count + kChunk - 1) / kChunk;
        if (index < n) {
            c = index;
            return true;
        }
        index -= n;
    }
    return false;
}
__device__ __forceinline__ size_t decay_at(const DecayedStateParams& p, uint32_t chunk, uint32_t a, bool channel) {
    return (size_t)p.chunks * p.heads * p.dim * p.vdim + ((size_t)chunk * p.heads + a) * (channel ? p.dim : 1);
}
// the sum over lanes `lane + 1 .. 63` (same-sign terms: a tree of additions, no subtraction)
__device__ __forceinline__ float suffix_after(float v, uint32_t lane) {
    float s = __shfl_down(v, 1, 64);
    s = lane < 63 ? s : 0.0f;
#pragma unroll
    for (int off = 1; off < 64; off <<= 1) {
        const float o = __shfl_down(s, off, 64);
        s += lane + off < 64 ? o : 0.0f;
    }
    return s;
}

// a workgroup per (chunk, head, tile of 64 key channels x 128 value columns): v_mfma_f32_32x32x2_f32, lane l feeds A[l % 32][k = l / 32], B[k = l / 32][l % 32] and holds
// rows 8 (r / 4) + 4 (l / 32) + r % 4 of column l % 32
template <bool CHANNEL>
__global__ void __launch_bounds__(256) decayed_state_local_kernel(DecayedStateParams p, float* ws) {
    constexpr uint32_t KW = 64, VW = 128;
    __shared__ float s_k[kChunk][KW], s_v[kChunk][VW], s_tot[4][KW]; // s_k: a decay per channel -- first the log decays
    __shared__ float s_e[kChunk];                                    // one decay per head: a row's step size times the decay behind it
    uint32_t z, c;
    SeqSpan sp;
    if (!find_chunk(p, blockIdx.x, z, c, sp)) return;
    const uint32_t a = blockIdx.y, g = a / (p.heads / p.groups), tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, l32 = lane & 31, half = lane >> 5;
    const uint32_t vtiles = (p.vdim + VW - 1) / VW, i0 = blockIdx.z / vtiles * KW, j0 = blockIdx.z % vtiles * VW;
    const uint32_t r0 = sp.row0 + c * kChunk, n = sp.count - c * kChunk < kChunk ? sp.count - c * kChunk : kChunk;
    if (!CHANNEL && wave == 0) { // lane = row: the decay of everything behind it
        const float dt = lane < n ? head_step(p, r0 + lane, a) : 0.0f;
        const float e = -expf(p.a_log[a]) * dt, behind = suffix_after(e, lane);
        s_e[lane] = dt * expf(behind);
        if (lane == 0 && blockIdx.z == 0) ws[decay_at(p, blockIdx.x, a, false)] = expf(e + behind);
    }
    if (CHANNEL)
        for (uint32_t e = tid; e < kChunk * KW; e += 256) {
            const uint32_t t = e / KW, i = e % KW;
            s_k[t][i] = (t < n && i0 + i < p.dim) ? channel_log_decay(p, r0 + t, a, i0 + i) : 0.0f;
        }
    for (uint32_t e = tid; e < kChunk * VW; e += 256) {
        const uint32_t t = e / VW, j = e % VW;
        s_v[t][j] = (t < n && j0 + j < p.vdim) ? p.rows_in[(size_t)(r0 + t) * p.ld + p.v_col + (size_t)a * p.vdim + j0 + j] : 0.0f;
    }
    __syncthreads();
    if (CHANNEL) { // thread = (channel, block of 16 rows)
        const uint32_t i = tid & 63, b = tid >> 6;
        float tot = 0.0f;
#pragma unroll
        for (uint32_t t = 0; t < kBlock; ++t) tot += s_k[b * kBlock + t][i];
        s_tot[b][i] = tot;
        __syncthreads();
        float behind = 0.0f;
        for (uint32_t o = 3; o > b; --o) behind += s_tot[o][i];
        if (b == 0 && j0 == 0 && i0 + i < p.dim) ws[decay_at(p, blockIdx.x, a, true) + i0 + i] = expf(behind + s_tot[0][i]);
        const float* kcol = p.rows_in + p.k_col + (size_t)g * p.dim + i0 + i;
#pragma unroll 4
        for (int t = kBlock - 1; t >= 0; --t) {
            const uint32_t row = b * kBlock + t;
            const float e = s_k[row][i];
            s_k[row][i] = (row < n && i0 + i < p.dim) ? kcol[(size_t)(r0 + row) * p.ld] * expf(behind) : 0.0f;
            behind += e;
        }
    } else {
        for (uint32_t e = tid; e < kChunk * KW; e += 256) {
            const uint32_t t = e / KW, i = e % KW;
            s_k[t][i] = (t < n && i0 + i < p.dim) ? p.rows_in[(size_t)(r0 + t) * p.ld + p.k_col + (size_t)g * p.dim + i0 + i] * s_e[t] : 0.0f;
        }
    }
    __syncthreads();
    // eight 32 x 32 tiles: wave w owns channel half w / 2 and column tiles 2 (w % 2), 2 (w % 2) + 1
    f32x16_m acc[2];
#pragma unroll
    for (int q = 0; q < 2; ++q)
#pragma unroll
        for (int r = 0; r < 16; ++r) acc[q][r] = 0.0f;
    const uint32_t ti = (wave >> 1) * 32, tj = (wave & 1) * 64, steps = (n + 1) / 2;
    if (i0 + ti < p.dim && j0 + tj < p.vdim) {
        for (uint32_t t2 = 0; t2 < steps; ++t2) {
            const uint32_t t = 2 * t2 + half;
            const float ka = s_k[t][ti + l32];
#pragma unroll
            for (int q = 0; q < 2; ++q) acc[q] = __builtin_amdgcn_mfma_f32_32x32x2f32(ka, s_v[t][tj + 32 * q + l32], acc[q], 0, 0, 0);
        }
        float* dst = ws + ((size_t)blockIdx.x * p.heads + a) * p.dim * p.vdim;
#pragma unroll
        for (int q = 0; q < 2; ++q) {
            const uint32_t j = j0 + tj + 32 * q + l32;
#pragma unroll
            for (int r = 0; r < 16; ++r) {
                const uint32_t i = i0 + ti + 8 * (r >> 2) + 4 * half + (r & 3);
                if (i < p.dim && j < p.vdim) dst[(size_t)i * p.vdim + j] = acc[q][r];
            }
        }
    }
}

// thread = state element; eight chunks' blocks are loaded ahead of the first of them that is replaced
template <bool CHANNEL> __global__ void __launch_bounds__(256) decayed_state_scan_kernel(DecayedStateParams p, float* ws) {
    constexpr uint32_t AHEAD = 8;
    const uint32_t z = blockIdx.x, a = blockIdx.y, elems = p.dim * p.vdim, e = blockIdx.z * 256 + threadIdx.x;
    const SeqSpan sp = p.spans[z];
    if (!sp.count || e >= elems) return;
    uint32_t first = 0; // the sequence's first chunk among the pass's chunks
    for (uint32_t q = 0; q < z; ++q) first += (p.spans[q].count + kChunk - 1) / kChunk;
    const uint32_t chunks = (sp.count + kChunk - 1) / kChunk, i = e / p.vdim;
    float* state = p.states[z] + (size_t)a * elems + e;
    float* slot = ws + ((size_t)first * p.heads + a) * elems + e;
    const float* dec = ws + decay_at(p, first, a, CHANNEL) + (CHANNEL ? i : 0);
    const size_t slot_step = (size_t)p.heads * elems, dec_step = (size_t)p.heads * (CHANNEL ? p.dim : 1);
    float S = sp.start ? *state : 0.0f;
    for (uint32_t c0 = 0; c0 < chunks; c0 += AHEAD) {
        float local[AHEAD], d[AHEAD];
#pragma unroll
        for (uint32_t u = 0; u < AHEAD; ++u) {
            const bool in = c0 + u < chunks;
            local[u] = in ? slot[(c0 + u) * slot_step] : 0.0f;
            d[u] = in ? dec[(c0 + u) * dec_step] : 0.0f;
        }
#pragma unroll
        for (uint32_t u = 0; u < AHEAD; ++u) {
            if (c0 + u >= chunks) break;
            slot[(c0 + u) * slot_step] = S;
            S = fmaf(d[u], S, local[u]);
        }
    }
    *state = S;
}

// a workgroup per (chunk, head, 128 value columns).  Key channels in slabs of 32: raw and decayed queries / keys in LDS; a wave owns the block of 16 x 16 scores on
// the diagonal that bears its number (running products, lane = (key row, quarter of the slab)), up to two of the six blocks below it (v_mfma_f32_16x16x4_f32) and,
// for the carried state, 32 rows x 64 columns of the result.
template <bool CHANNEL>
__global__ void __launch_bounds__(256) decayed_state_out_kernel(DecayedStateParams p, const float* ws) {
    constexpr uint32_t SW = 32, PW = SW + 4, VW = 128; // a slab row's pitch: 16-byte aligned, rows on distinct banks
    constexpr uint32_t ROWS = kChunk * PW;
    __shared__ __attribute__((aligned(16))) float s_buf[CHANNEL ? 5 * ROWS : (2 * ROWS + kChunk * PW > kChunk * VW ? 2 * ROWS + kChunk * PW : kChunk * VW)];
    __shared__ float s_p[kChunk][kChunk + 1], s_tot[4][SW]; // s_tot: a block's whole decay per channel of the slab
    __shared__ float s_h[3][kChunk]; // one decay per head: log decays, step sizes, the decay from the chunk's start up to and including a row
    uint32_t z, c;
    SeqSpan sp;
    if (!find_chunk(p, blockIdx.x, z, c, sp)) return;
    const uint32_t a = blockIdx.y, g = a / (p.heads / p.groups), tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, l32 = lane & 31, half = lane >> 5, l16 = lane & 15, quarter = lane >> 4;
    const uint32_t j0 = blockIdx.z * VW, dim = p.dim, vdim = p.vdim;
    const uint32_t r0 = sp.row0 + c * kChunk, n = sp.count - c * kChunk < kChunk ? sp.count - c * kChunk : kChunk;
    const float* base = p.rows_in + (size_t)r0 * p.ld;
    const float *qb = base + p.q_col + (size_t)g * dim, *kb = base + p.k_col + (size_t)g * dim;
    const bool carried = sp.start || c;
    const float* S = ws + ((size_t)blockIdx.x * p.heads + a) * dim * vdim + j0;
    float *s_q = s_buf, *s_k = s_buf + ROWS, *s_x = s_buf + 2 * ROWS; // s_x: one decay per head -- queries decayed from the chunk's start
    float *s_e = s_buf + 2 * ROWS, *s_qd = s_buf + 3 * ROWS, *s_kd = s_buf + 4 * ROWS; // a decay per channel: decays; queries decayed from their block's start; keys decayed to its end
    for (uint32_t e = tid; e < kChunk * (kChunk + 1); e += 256) (&s_p[0][0])[e] = 0.0f;
    if (!CHANNEL) {
        if (wave == 0) {
            const float dt = lane < n ? head_step(p, r0 + lane, a) : 0.0f, e = -expf(p.a_log[a]) * dt;
            float upto = e; // the sum over lanes 0 .. lane
#pragma unroll
            for (int off = 1; off < 64; off <<= 1) {
                const float o = __shfl_up(upto, off, 64);
                upto += lane >= (uint32_t)off ? o : 0.0f;
            }
            s_h[0][lane] = e, s_h[1][lane] = dt, s_h[2][lane] = expf(upto);
        }
        __syncthreads();
        // thread = (key row j, block of 16 query rows): e^(the log decays of rows j + 1 .. i), summed from j on
        const uint32_t j = lane, b = wave;
        float sum = 0.0f;
        const uint32_t i_lo = b * kBlock;
        for (uint32_t t = j + 1; t < i_lo; ++t) sum += s_h[0][t];
        const float dt = s_h[1][j];
        for (uint32_t i = i_lo; i < i_lo + kBlock; ++i) {
            if (i < j) continue;
            if (i > j) sum += s_h[0][i];
            s_p[i][j] = i < n ? expf(sum) * dt : 0.0f;
        }
    }
    const uint32_t pi = wave >> 1, pj = wave & 1; // 32-row half of the result; one decay per head: 32-column half of the scores; result column tiles 2 pj, 2 pj + 1
    f32x16_m sc, o[2];
#pragma unroll
    for (int r = 0; r < 16; ++r) sc[r] = 0.0f, o[0][r] = 0.0f, o[1][r] = 0.0f;
    // the six pairs of blocks below the diagonal: (1, 0), (2, 0), (2, 1), (3, 0), (3, 1), (3, 2)
    auto below_i = [](uint32_t pair) { return pair < 1 ? 1u : pair < 3 ? 2u : 3u; };
    auto below_j = [&](uint32_t pair) { const uint32_t i = below_i(pair); return pair - i * (i - 1) / 2; };
    f32x4_m lower[2] = {{0.f, 0.f, 0.f, 0.f}, {0.f, 0.f, 0.f, 0.f}};
    float diag[kBlock];
#pragma unroll
    for (uint32_t i = 0; i < kBlock; ++i) diag[i] = 0.0f;
    const bool out_on = j0 + pj * 64 < vdim;
    for (uint32_t d0 = 0; d0 < dim; d0 += SW) {
        __syncthreads(); // the slab before has been read
        for (uint32_t e = tid; e < kChunk * SW; e += 256) {
            const uint32_t r = e / SW, dd = e % SW, d = d0 + dd;
            const bool ok = r < n && d < dim;
            const float q = ok ? qb[(size_t)r * p.ld + d] * p.q_scale : 0.0f;
            s_q[r * PW + dd] = q;
            s_k[r * PW + dd] = ok ? kb[(size_t)r * p.ld + d] : 0.0f;
            if (CHANNEL) s_e[r * PW + dd] = ok ? channel_log_decay(p, r0 + r, a, d) : 0.0f;
            else s_x[r * PW + dd] = q * s_h[2][r];
        }
        __syncthreads();
        if (CHANNEL) { // thread = (channel, block, direction): prefixes onto the queries, suffixes onto the keys; the log decays become decays behind them
            const uint32_t dd = tid & 31, b = (tid >> 5) & 3, first = b * kBlock;
            float sum = 0.0f;
            if (tid < 128) {
#pragma unroll 4
                for (uint32_t t = 0; t < kBlock; ++t) {
                    sum += s_e[(first + t) * PW + dd];
                    s_qd[(first + t) * PW + dd] = s_q[(first + t) * PW + dd] * expf(sum);
                }
                s_tot[b][dd] = expf(sum);
            } else {
#pragma unroll 4
                for (int t = kBlock - 1; t >= 0; --t) {
                    s_kd[(first + t) * PW + dd] = s_k[(first + t) * PW + dd] * expf(sum);
                    sum += s_e[(first + t) * PW + dd];
                }
            }
            __syncthreads();
            for (uint32_t e = tid; e < kChunk * SW; e += 256) s_e[e / SW * PW + e % SW] = expf(s_e[e / SW * PW + e % SW]);
            __syncthreads();
            {   // the diagonal block `wave`: key row l16, channels 8 quarter .. 8 quarter + 7 of the slab
                const uint32_t first_row = wave * kBlock, ch = quarter * 8;
                float w[8];
                const f32x4_m k0 = *(const f32x4_m*)(s_k + (first_row + l16) * PW + ch), k1 = *(const f32x4_m*)(s_k + (first_row + l16) * PW + ch + 4);
#pragma unroll
                for (int u = 0; u < 4; ++u) w[u] = k0[u], w[u + 4] = k1[u];
#pragma unroll
                for (uint32_t i = 0; i < kBlock; ++i) {
                    const float* er = s_e + (first_row + i) * PW + ch;
                    const float* qr = s_q + (first_row + i) * PW + ch;
                    const f32x4_m e0 = *(const f32x4_m*)er, e1 = *(const f32x4_m*)(er + 4), q0 = *(const f32x4_m*)qr, q1 = *(const f32x4_m*)(qr + 4);
                    float dot = 0.0f;
#pragma unroll
                    for (int u = 0; u < 8; ++u) {
                        const float ev = u < 4 ? e0[u] : e1[u - 4], qv = u < 4 ? q0[u] : q1[u - 4];
                        w[u] = i > l16 ? w[u] * ev : w[u];
                        dot = fmaf(qv, w[u], dot);
                    }
                    diag[i] += i >= l16 ? dot : 0.0f;
                }
            }
#pragma unroll
            for (int q = 0; q < 2; ++q) { // blocks below the diagonal: whole blocks in between decay the query operand
                const uint32_t pair = wave + 4 * q;
                if (pair >= 6) continue;
                const uint32_t bi = below_i(pair), bj = below_j(pair);
#pragma unroll
                for (uint32_t k4 = 0; k4 < SW; k4 += 4) {
                    const uint32_t ch = k4 + quarter;
                    float qa = s_qd[(bi * kBlock + l16) * PW + ch];
                    for (uint32_t b = bj + 1; b < bi; ++b) qa *= s_tot[b][ch];
                    lower[q] = __builtin_amdgcn_mfma_f32_16x16x4f32(qa, s_kd[(bj * kBlock + l16) * PW + ch], lower[q], 0, 0, 0);
                }
            }
        } else {
#pragma unroll 4
            for (uint32_t d = 0; d < SW; d += 2) sc = __builtin_amdgcn_mfma_f32_32x32x2f32(s_q[(pi * 32 + l32) * PW + d + half], s_k[(pj * 32 + l32) * PW + d + half], sc, 0, 0, 0);
        }
        if (carried && out_on) { // + sum_d (query decayed from the chunk's start) S[d][column], the state's rows straight from memory
#pragma unroll 4
            for (uint32_t d = 0; d < SW; d += 2) {
                const uint32_t dl = d + half, dg = d0 + dl, row = pi * 32 + l32;
                float qa;
                if (CHANNEL) {
                    qa = s_qd[row * PW + dl];
                    for (uint32_t b = 0; b < row / kBlock; ++b) qa *= s_tot[b][dl];
                } else {
                    qa = s_x[row * PW + dl];
                }
#pragma unroll
                for (int q = 0; q < 2; ++q) {
                    const uint32_t col = pj * 64 + 32 * q + l32;
                    const float sv = (dg < dim && j0 + col < vdim) ? S[(size_t)dg * vdim + col] : 0.0f;
                    o[q] = __builtin_amdgcn_mfma_f32_32x32x2f32(qa, sv, o[q], 0, 0, 0);
                }
            }
        }
    }
    __syncthreads(); // the slabs are done with
    if (CHANNEL) {
#pragma unroll
        for (uint32_t i = 0; i < kBlock; ++i) {
            float v = diag[i];
            v += __shfl_xor(v, 16, 64);
            v += __shfl_xor(v, 32, 64);
            if (quarter == 0 && i >= l16) s_p[wave * kBlock + i][wave * kBlock + l16] = v;
        }
#pragma unroll
        for (int q = 0; q < 2; ++q) {
            const uint32_t pair = wave + 4 * q;
            if (pair >= 6) continue;
#pragma unroll
            for (int r = 0; r < 4; ++r) s_p[below_i(pair) * kBlock + 4 * quarter + r][below_j(pair) * kBlock + l16] = lower[q][r];
        }
    } else {
#pragma unroll
        for (int r = 0; r < 16; ++r) { // (above the diagonal and beyond the chunk's rows s_p holds zeros)
            const uint32_t i = pi * 32 + 8 * (r >> 2) + 4 * half + (r & 3), j = pj * 32 + l32;
            s_p[i][j] *= sc[r];
        }
    }
    float* s_v = s_buf; // [64][VW]
    for (uint32_t e = tid; e < kChunk * VW; e += 256) {
        const uint32_t t = e / VW, j = e % VW;
        s_v[e] = (t < n && j0 + j < vdim) ? base[(size_t)t * p.ld + p.v_col + (size_t)a * vdim + j0 + j] : 0.0f;
    }
    __syncthreads();
    if (!out_on) return;
    const uint32_t last = n < pi * 32 + 32 ? n : pi * 32 + 32, steps = (last + 1) / 2; // keys up to this half's last row
    for (uint32_t t2 = 0; t2 < steps; ++t2) {
        const uint32_t t = 2 * t2 + half;
        const float pa = s_p[pi * 32 + l32][t];
#pragma unroll
        for (int q = 0; q < 2; ++q) o[q] = __builtin_amdgcn_mfma_f32_32x32x2f32(pa, s_v[t * VW + pj * 64 + 32 * q + l32], o[q], 0, 0, 0);
    }
    const float skip = p.skip ? p.skip[a] : 0.0f;
#pragma unroll
    for (int q = 0; q < 2; ++q) {
        const uint32_t col = pj * 64 + 32 * q + l32;
        if (j0 + col >= vdim) continue;
#pragma unroll
        for (int r = 0; r < 16; ++r) {
            const uint32_t i = pi * 32 + 8 * (r >> 2) + 4 * half + (r & 3);
            if (i < n) p.out[((size_t)(r0 + i) * p.heads + a) * vdim + j0 + col] = p.skip ? fmaf(skip, s_v[i * VW + col], o[q][r]) : o[q][r];
        }
    }
}

} // namespace

size_t decayed_state_chunk_ws_bytes(uint32_t chunks, uint32_t heads, uint32_t dim, uint32_t vdim) { return (size_t)chunks * heads * ((size_t)dim * vdim + dim) * 4; }

bool decayed_state_supported(uint32_t dim, uint32_t vdim) { return dim >= 1 && dim <= 1024 && vdim >= 1 && vdim <= 65536; }

uzu_status decayed_state(hipStream_t s, const DecayedStateParams& p) {
    if (!p.rows || !p.nseq) return UZU_OK;
    UZU_REQUIRE(p.rows_in && p.decay && p.out && p.states && p.spans && p.heads && p.groups && p.heads % p.groups == 0, "decayed_state: null argument");
    UZU_REQUIRE(p.per_head ? (p.a_log && p.dt_bias) : p.inv_temperature > 0.0f, "decayed_state: the decays' constants");
    UZU_UNSUPPORTED(!decayed_state_supported(p.dim, p.vdim), "decayed_state: heads of %u x %u (keys up to 1024)", p.dim, p.vdim);
    UZU_REQUIRE((size_t)p.nseq * p.heads <= 0x7FFFFFFFu && p.heads <= 65535 && p.nseq <= 65535, "decayed_state: too many heads for one launch");
    if (p.form == 2 || (p.form == 0 && p.chunk_ws && p.rows > 16 * p.nseq)) { // prompt-sized: in chunks
        UZU_REQUIRE(p.chunk_ws && p.chunks && p.chunk_ws_bytes >= decayed_state_chunk_ws_bytes(p.chunks, p.heads, p.dim, p.vdim), "decayed_state: the chunked form needs its workspace");
        const uint32_t vt = (p.vdim + 127) / 128, kt = (p.dim + 63) / 64;
        UZU_REQUIRE((size_t)vt * kt <= 65535 && ((size_t)p.dim * p.vdim + 255) / 256 <= 65535, "decayed_state: head widths %u x %u", p.dim, p.vdim);
        const dim3 lgrid(p.chunks, p.heads, vt * kt), sgrid(p.nseq, p.heads, (uint32_t)(((size_t)p.dim * p.vdim + 255) / 256)), ogrid(p.chunks, p.heads, vt);
        float* ws = p.chunk_ws;
        if (p.per_head) {
            UZU_PROPAGATE(launch_check([&] { hipLaunchKernelGGL(decayed_state_local_kernel<false>, lgrid, dim3(256), 0, s, p, ws); }, "decayed_state_local"));
            UZU_PROPAGATE(launch_check([&] { hipLaunchKernelGGL(decayed_state_scan_kernel<false>, sgrid, dim3(256), 0, s, p, ws); }, "decayed_state_scan"));
            return launch_check([&] { hipLaunchKernelGGL(decayed_state_out_kernel<false>, ogrid, dim3(256), 0, s, p, (const float*)ws); }, "decayed_state_out");
        }
        UZU_PROPAGATE(launch_check([&] { hipLaunchKernelGGL(decayed_state_local_kernel<true>, lgrid, dim3(256), 0, s, p, ws); }, "decayed_state_local"));
        UZU_PROPAGATE(launch_check([&] { hipLaunchKernelGGL(decayed_state_scan_kernel<true>, sgrid, dim3(256), 0, s, p, ws); }, "decayed_state_scan"));
        return launch_check([&] { hipLaunchKernelGGL(decayed_state_out_kernel<true>, ogrid, dim3(256), 0, s, p, (const float*)ws); }, "decayed_state_out");
    }
    const dim3 grid(p.nseq * p.heads, (p.vdim + 15) / 16);
#define UZU_DS(N)                                                                                                                                                     \
    do {                                                                                                                                                              \
        if (p.per_head) return launch_check([&] { hipLaunchKernelGGL((decayed_state_steps_kernel<N, false>), grid, dim3(256), 0, s, p); }, "decayed_state_steps");    \
        return launch_check([&] { hipLaunchKernelGGL((decayed_state_steps_kernel<N, true>), grid, dim3(256), 0, s, p); }, "decayed_state_steps");                     \
    } while (0)
    if (p.dim <= 32) UZU_DS(2);
    if (p.dim <= 64) UZU_DS(4);
    if (p.dim <= 128) UZU_DS(8);
    if (p.dim <= 256) UZU_DS(16);
    if (p.dim <= 512) UZU_DS(32);
    UZU_DS(64);
#undef UZU_DS
}

} // namespace k
} // namespace uzu
