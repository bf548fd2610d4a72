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

__device__ __forceinline__ float softplus_f32(float z) { return fmaxf(z, 0.0f) + log1pf(expf(-fabsf(z))); }

// one decay per head: the step size of a row (it multiplies the key); the row's log decay is -exp(a_log) times it
__device__ __forceinline__ float head_step(const DecayedStateParams& p, uint32_t r, uint32_t a) { return softplus_f32(p.decay[(size_t)r * p.lddecay + a] + p.dt_bias[a]); }
// a decay per key channel: sigmoid(z)^inv_temperature by way of its logarithm, min(z, 0) - ln(1 + e^(-|z|)) (an absolute error of one rounding of 1: what the decay
// itself is rounded to)
__device__ __forceinline__ float channel_decay(float z, float inv_temperature) { return fast_exp((fminf(z, 0.0f) - fast_log(1.0f + fast_exp(-fabsf(z)))) * inv_temperature); }

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
            if (CHANNEL) s_e[c] = in ? channel_decay(p.decay[(size_t)r * p.lddecay + (size_t)a * p.dim + c], p.inv_temperature) : 0.0f;
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
// the sum over a quad of lanes, left in every one of them
__device__ __forceinline__ float quad_sum(float v) {
    v += __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, v), 0xB1, 0xF, 0xF, true)); // quad_perm [1, 0, 3, 2]
    v += __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, v), 0x4E, 0xF, 0xF, true)); // quad_perm [2, 3, 0, 1]
    return v;
}
// four neighbouring floats of a row, those from `left` on zero; aligned: one 16-byte load (the host has checked pitch, columns and widths)
__device__ __forceinline__ f32x4_m load4(const float* at, uint32_t left, bool aligned) {
    f32x4_m v{0.f, 0.f, 0.f, 0.f};
    if (aligned) {
        if (left) v = *(const f32x4_m*)at;
    } else {
#pragma unroll
        for (uint32_t u = 0; u < 4; ++u)
            if (u < left) v[u] = at[u];
    }
    return v;
}

// a workgroup per (chunk, head, tile of 64 key channels x 64 NQ value columns): v_mfma_f32_32x32x2_f32, lane l feeds A[l % 32][k = l / 32], B[k = l / 32][l % 32] and
// holds rows 8 (r / 4) + 4 (l / 32) + r % 4 of column l % 32
template <bool CHANNEL, int NQ>
__global__ void __launch_bounds__(256) decayed_state_local_kernel(DecayedStateParams p, float* ws, uint32_t aligned) {
    constexpr uint32_t KW = 64, VW = 64 * NQ;
    __shared__ __attribute__((aligned(16))) float s_k[kChunk][KW], s_v[kChunk][VW];
    __shared__ float s_tot[4][KW]; // a decay per channel: a block's whole decay
    __shared__ float s_e[kChunk];  // one decay per head: a row's step size times the decay behind it
    uint32_t z, c;
    SeqSpan sp;
    if (!find_chunk(p, blockIdx.x, z, c, sp)) return;
    const uint32_t a = blockIdx.y, g = a / (p.heads / p.groups), tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, l32 = lane & 31, half = lane >> 5;
    const uint32_t vtiles = (p.vdim + VW - 1) / VW, i0 = blockIdx.z / vtiles * KW, j0 = blockIdx.z % vtiles * VW;
    const uint32_t r0 = sp.row0 + c * kChunk, n = sp.count - c * kChunk < kChunk ? sp.count - c * kChunk : kChunk;
    // thread = (channel i of the tile, block b of 16 rows): its keys (and decays) in registers, every load in front of the first use
    const uint32_t i = lane, b = wave;
    const bool in = i0 + i < p.dim;
    const float* kcol = p.rows_in + (size_t)r0 * p.ld + p.k_col + (size_t)g * p.dim + i0 + i;
    float key[kBlock], dec[CHANNEL ? kBlock : 1];
#pragma unroll
    for (uint32_t t = 0; t < kBlock; ++t) {
        const uint32_t row = b * kBlock + t;
        key[t] = row < n && in ? kcol[(size_t)row * p.ld] : 0.0f;
        if (CHANNEL) dec[CHANNEL ? t : 0] = row < n && in ? p.decay[(size_t)(r0 + row) * p.lddecay + (size_t)a * p.dim + i0 + i] : 0.0f;
    }
    {   // values: thread = (rows tid / (16 NQ) + .., four columns)
        constexpr uint32_t TPR = 16 * NQ, RPP = 256 / TPR;
        const uint32_t col = (tid % TPR) * 4, left = j0 + col < p.vdim ? p.vdim - j0 - col : 0;
        const float* vb = p.rows_in + (size_t)r0 * p.ld + p.v_col + (size_t)a * p.vdim + j0 + col;
        f32x4_m v[kChunk / RPP];
#pragma unroll
        for (uint32_t u = 0; u < kChunk / RPP; ++u) {
            const uint32_t t = tid / TPR + u * RPP;
            v[u] = load4(vb + (size_t)t * p.ld, t < n ? left : 0, aligned);
        }
#pragma unroll
        for (uint32_t u = 0; u < kChunk / RPP; ++u) *(f32x4_m*)&s_v[tid / TPR + u * RPP][col] = v[u];
    }
    if (CHANNEL) {
        float run = 1.0f; // the decay of the rows behind t inside the block
#pragma unroll
        for (int t = kBlock - 1; t >= 0; --t) {
            key[t] *= run;
            run *= b * kBlock + t < n ? channel_decay(dec[CHANNEL ? t : 0], p.inv_temperature) : 1.0f;
        }
        s_tot[b][i] = run;
        __syncthreads();
        float behind = 1.0f;
        for (uint32_t o = b + 1; o < 4; ++o) behind *= s_tot[o][i];
        if (b == 0 && j0 == 0 && in) ws[decay_at(p, blockIdx.x, a, true) + i0 + i] = run * behind;
#pragma unroll
        for (uint32_t t = 0; t < kBlock; ++t) s_k[b * kBlock + t][i] = key[t] * behind;
    } else {
        if (wave == 0) { // lane = row: its step size and the decay of everything behind it
            const float dt = lane < n ? head_step(p, r0 + lane, a) : 0.0f;
            const float e = -expf(p.a_log[a]) * dt, behind = suffix_after(e, lane);
            s_e[lane] = dt * expf(behind);
            if (lane == 0 && blockIdx.z == 0) ws[decay_at(p, blockIdx.x, a, false)] = expf(e + behind);
        }
        __syncthreads();
#pragma unroll
        for (uint32_t t = 0; t < kBlock; ++t) s_k[b * kBlock + t][i] = key[t] * s_e[b * kBlock + t];
    }
    __syncthreads();
    // 32 x 32 tiles: wave w owns channel half w / 2 and column tiles NQ (w % 2) ..
    f32x16_m acc[NQ];
#pragma unroll
    for (int q = 0; q < NQ; ++q)
#pragma unroll
        for (int r = 0; r < 16; ++r) acc[q][r] = 0.0f;
    const uint32_t ti = (wave >> 1) * 32, tj = (wave & 1) * 32 * NQ;
    if (i0 + ti >= p.dim || j0 + tj >= p.vdim) return;
    for (uint32_t t0 = 0; t0 < n; t0 += 8) // (rows beyond the chunk's: zero keys and values)
#pragma unroll
        for (uint32_t u = 0; u < 4; ++u) {
            const uint32_t t = t0 + 2 * u + half;
            const float ka = s_k[t][ti + l32];
#pragma unroll
            for (int q = 0; q < NQ; ++q) acc[q] = __builtin_amdgcn_mfma_f32_32x32x2f32(ka, s_v[t][tj + 32 * q + l32], acc[q], 0, 0, 0);
        }
    float* dst = ws + ((size_t)blockIdx.x * p.heads + a) * p.dim * p.vdim;
#pragma unroll
    for (int q = 0; q < NQ; ++q) {
        const uint32_t j = j0 + tj + 32 * q + l32;
#pragma unroll
        for (int r = 0; r < 16; ++r) {
            const uint32_t row = i0 + ti + 8 * (r >> 2) + 4 * half + (r & 3);
            if (row < p.dim && j < p.vdim) dst[(size_t)row * p.vdim + j] = acc[q][r];
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

// a workgroup per (chunk, head, 64 NQ value columns).  Key channels in slabs of 32; the next slab's rows travel from memory into registers while the current one is
// worked on, the carried state's rows go from memory straight into the products.  One decay per head: scores as two 32 x 32 tiles per wave row, times a table of decays.
// A decay per channel: a wave owns the block of 16 x 16 scores on the diagonal that bears its number (running products, lane = (key row, quarter of the slab)) and up to
// two of the six blocks below it (v_mfma_f32_16x16x4_f32).  Results: wave w has rows 32 (w / 2) .., column tiles NQ (w % 2) ..
template <bool CHANNEL, int NQ>
__global__ void __launch_bounds__(256, CHANNEL ? 2 : 3) decayed_state_out_kernel(DecayedStateParams p, const float* ws, uint32_t aligned) {
    constexpr uint32_t SW = 32, PW = SW + 4, VW = 64 * NQ, ROWS = kChunk * PW; // a slab row's pitch: 16-byte aligned, rows on distinct banks
    constexpr uint32_t BUF = CHANNEL ? 5 * ROWS : 2 * ROWS;
    __shared__ __attribute__((aligned(16))) float s_buf[BUF > kChunk * VW ? BUF : kChunk * VW];
    __shared__ float s_p[kChunk][kChunk + 1], s_tot[4][SW]; // s_tot: a block's whole decay per channel of the slab
    __shared__ float s_h[6][kChunk]; // one decay per head, by row: log decay, step size, decay from the chunk's start, sums of log decays up to the row / behind it in its block, blocks' sums
    uint32_t z, c;
    SeqSpan sp;
    if (!find_chunk(p, blockIdx.x, z, c, sp)) return;
    const uint32_t a = blockIdx.y, g = a / (p.heads / p.groups), tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, l32 = lane & 31, half = lane >> 5, l16 = lane & 15, quarter = lane >> 4;
    const uint32_t j0 = blockIdx.z * VW, dim = p.dim, vdim = p.vdim;
    const uint32_t r0 = sp.row0 + c * kChunk, n = sp.count - c * kChunk < kChunk ? sp.count - c * kChunk : kChunk;
    const float* base = p.rows_in + (size_t)r0 * p.ld;
    const float *qb = base + p.q_col + (size_t)g * dim, *kb = base + p.k_col + (size_t)g * dim, *eb = p.decay + (size_t)r0 * p.lddecay + (size_t)a * dim;
    const float* S = ws + ((size_t)blockIdx.x * p.heads + a) * dim * vdim + j0;
    float *s_q = s_buf, *s_k = s_buf + ROWS;
    float *s_e = s_buf + 2 * ROWS, *s_qd = s_buf + 3 * ROWS, *s_kd = s_buf + 4 * ROWS; // a decay per channel: decays; queries decayed from their block's start; keys decayed to its end
    const uint32_t pi = wave >> 1, pj = wave & 1;
    const bool out_on = j0 + pj * 32 * NQ < vdim, carried = (sp.start || c) && out_on;
    // a slab's loads: thread = (rows tid / 8, tid / 8 + 32, four channels)
    const uint32_t lr = tid >> 3, lc = (tid & 7) * 4;
    f32x4_m fq[2], fk[2], fe[CHANNEL ? 2 : 1];
    auto fetch = [&](uint32_t d0) {
        const uint32_t left = d0 + lc < dim ? dim - d0 - lc : 0;
#pragma unroll
        for (uint32_t u = 0; u < 2; ++u) {
            const uint32_t r = lr + 32 * u, m = r < n ? left : 0;
            fq[u] = load4(qb + (size_t)r * p.ld + d0 + lc, m, aligned);
            fk[u] = load4(kb + (size_t)r * p.ld + d0 + lc, m, aligned);
            if (CHANNEL) fe[CHANNEL ? u : 0] = load4(eb + (size_t)r * p.lddecay + d0 + lc, m, aligned);
        }
    };
    fetch(0);
    if (!CHANNEL) {
        for (uint32_t e = tid; e < kChunk * (kChunk + 1); e += 256) (&s_p[0][0])[e] = 0.0f;
        if (wave == 0) {
            const float dt = lane < n ? head_step(p, r0 + lane, a) : 0.0f, e = -expf(p.a_log[a]) * dt;
            float upto = e, behind = __shfl_down(e, 1, 16); // inside the row's block of 16
            behind = l16 < 15 ? behind : 0.0f;
#pragma unroll
            for (int off = 1; off < 16; off <<= 1) {
                const float o = __shfl_up(upto, off, 16), q = __shfl_down(behind, off, 16);
                upto += l16 >= (uint32_t)off ? o : 0.0f;
                behind += l16 + off < 16 ? q : 0.0f;
            }
            const float tot = __shfl(upto, 15, 16);
            float before = 0.0f; // the blocks in front
#pragma unroll
            for (uint32_t o = 0; o < 3; ++o) {
                const float t = __shfl(tot, (int)(o * kBlock), 64);
                before += o < quarter ? t : 0.0f;
            }
            s_h[0][lane] = e, s_h[1][lane] = dt, s_h[2][lane] = expf(before + upto), s_h[3][lane] = upto, s_h[4][lane] = behind, s_h[5][quarter] = tot;
        }
        __syncthreads();
        // thread = (key row j, block of 16 query rows): step_j e^(the log decays of rows j + 1 .. i)
        const uint32_t j = lane, b = wave, jb = j / kBlock;
        const float dt = s_h[1][j];
        if (b > jb) {
            float sum = s_h[4][j];
            for (uint32_t o = jb + 1; o < b; ++o) sum += s_h[5][o];
#pragma unroll 4
            for (uint32_t i = b * kBlock; i < b * kBlock + kBlock; ++i) s_p[i][j] = i < n ? expf(sum + s_h[3][i]) * dt : 0.0f;
        } else if (b == jb) {
            float sum = 0.0f;
#pragma unroll 4
            for (uint32_t i = b * kBlock; i < b * kBlock + kBlock; ++i) {
                sum += i > j ? s_h[0][i] : 0.0f;
                if (i >= j) s_p[i][j] = i < n ? expf(sum) * dt : 0.0f;
            }
        }
    } else {
        for (uint32_t e = tid; e < kChunk * (kChunk + 1); e += 256) (&s_p[0][0])[e] = 0.0f;
    }
    f32x16_m sc, o[NQ];
#pragma unroll
    for (int r = 0; r < 16; ++r) sc[r] = 0.0f;
#pragma unroll
    for (int q = 0; q < NQ; ++q)
#pragma unroll
        for (int r = 0; r < 16; ++r) o[q][r] = 0.0f;
    // the six pairs of blocks below the diagonal: (1, 0), (2, 0), (2, 1), (3, 0), (3, 1), (3, 2)
    auto below_i = [](uint32_t pair) { return pair < 1 ? 1u : pair < 3 ? 2u : 3u; };
    auto below_j = [&](uint32_t pair) { const uint32_t i = below_i(pair); return pair - i * (i - 1) / 2; };
    f32x4_m lower[2] = {{0.f, 0.f, 0.f, 0.f}, {0.f, 0.f, 0.f, 0.f}};
    const uint32_t row = pi * 32 + l32; // this lane's row of the query operand
    float from_start = 1.0f;
    for (uint32_t d0 = 0; d0 < dim; d0 += SW) {
        float sv[SW / 2][NQ]; // the carried state's rows of the slab
#pragma unroll
        for (uint32_t d = 0; d < SW / 2; ++d)
#pragma unroll
            for (int q = 0; q < NQ; ++q) {
                const uint32_t dg = d0 + 2 * d + half, col = pj * 32 * NQ + 32 * q + l32;
                sv[d][q] = carried && dg < dim && j0 + col < vdim ? S[(size_t)dg * vdim + col] : 0.0f;
            }
        __syncthreads(); // the slab before has been read
#pragma unroll
        for (uint32_t u = 0; u < 2; ++u) {
            const uint32_t at = (lr + 32 * u) * PW + lc;
            *(f32x4_m*)(s_q + at) = fq[u] * p.q_scale;
            *(f32x4_m*)(s_k + at) = fk[u];
            if (CHANNEL) { // (rows and channels beyond the chunk: their queries and keys are zeros)
                f32x4_m e;
#pragma unroll
                for (int v = 0; v < 4; ++v) e[v] = channel_decay(fe[CHANNEL ? u : 0][v], p.inv_temperature);
                *(f32x4_m*)(s_e + at) = e;
            }
        }
        __syncthreads();
        if (d0 + SW < dim) fetch(d0 + SW);
        if (CHANNEL) { // thread = (channel, block, direction): running products onto the queries from the block's start, onto the keys from its end
            const uint32_t dd = tid & 31, first = ((tid >> 5) & 3) * kBlock;
            float run = 1.0f;
            if (tid < 128) {
#pragma unroll
                for (uint32_t t = 0; t < kBlock; ++t) {
                    run *= s_e[(first + t) * PW + dd];
                    s_qd[(first + t) * PW + dd] = s_q[(first + t) * PW + dd] * run;
                }
                s_tot[first / kBlock][dd] = run;
            } else {
#pragma unroll
                for (int t = kBlock - 1; t >= 0; --t) {
                    s_kd[(first + t) * PW + dd] = s_k[(first + t) * PW + dd] * run;
                    run *= s_e[(first + t) * PW + dd];
                }
            }
            __syncthreads();
            {   // the diagonal block `wave`: four lanes share a key row, channels 8 quad .. 8 quad + 7 of the slab each; the sums gather in s_p
                const uint32_t first_row = wave * kBlock, j = lane >> 2, ch = (lane & 3) * 8;
                const f32x4_m k0 = *(const f32x4_m*)(s_k + (first_row + j) * PW + ch), k1 = *(const f32x4_m*)(s_k + (first_row + j) * PW + ch + 4);
                f32x4_m w0{0.f, 0.f, 0.f, 0.f}, w1 = w0; // the key as row i sees it: nothing in front of its own row
#pragma unroll 2
                for (uint32_t i = 0; i < kBlock; ++i) {
                    const float *er = s_e + (first_row + i) * PW + ch, *qr = s_q + (first_row + i) * PW + ch;
                    const f32x4_m e0 = *(const f32x4_m*)er, e1 = *(const f32x4_m*)(er + 4), q0 = *(const f32x4_m*)qr, q1 = *(const f32x4_m*)(qr + 4);
                    const bool own = i == j;
                    float d0v = 0.0f, d1v = 0.0f;
#pragma unroll
                    for (int u = 0; u < 4; ++u) {
                        w0[u] = own ? k0[u] : w0[u] * e0[u], w1[u] = own ? k1[u] : w1[u] * e1[u];
                        d0v = fmaf(q0[u], w0[u], d0v), d1v = fmaf(q1[u], w1[u], d1v);
                    }
                    const float dot = quad_sum(d0v + d1v);
                    if ((lane & 3) == 0) s_p[first_row + i][first_row + j] += dot;
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
                    if (bi - bj > 1) qa *= s_tot[bj + 1][ch];
                    if (bi - bj > 2) qa *= s_tot[bj + 2][ch];
                    lower[q] = __builtin_amdgcn_mfma_f32_16x16x4f32(qa, s_kd[(bj * kBlock + l16) * PW + ch], lower[q], 0, 0, 0);
                }
            }
            if (carried) { // + sum_d (query decayed from the chunk's start) S[d][column]
                const uint32_t rb = row / kBlock;
#pragma unroll
                for (uint32_t d = 0; d < SW / 2; ++d) {
                    const uint32_t dl = 2 * d + half;
                    float qa = s_qd[row * PW + dl];
                    const float t0 = s_tot[0][dl], t1 = s_tot[1][dl], t2 = s_tot[2][dl];
                    qa *= rb > 0 ? t0 : 1.0f;
                    qa *= rb > 1 ? t1 : 1.0f;
                    qa *= rb > 2 ? t2 : 1.0f;
#pragma unroll
                    for (int q = 0; q < NQ; ++q) o[q] = __builtin_amdgcn_mfma_f32_32x32x2f32(qa, sv[d][q], o[q], 0, 0, 0);
                    if ((d & 3) == 3) __builtin_amdgcn_sched_barrier(0);
                }
            }
        } else {
            if (d0 == 0) from_start = s_h[2][row];
#pragma unroll
            for (uint32_t d = 0; d < SW / 2; ++d) {
                const float qv = s_q[row * PW + 2 * d + half];
                sc = __builtin_amdgcn_mfma_f32_32x32x2f32(qv, s_k[(pj * 32 + l32) * PW + 2 * d + half], sc, 0, 0, 0);
                if (carried) {
#pragma unroll
                    for (int q = 0; q < NQ; ++q) o[q] = __builtin_amdgcn_mfma_f32_32x32x2f32(qv * from_start, sv[d][q], o[q], 0, 0, 0);
                }
            }
        }
    }
    __syncthreads(); // the slabs are done with
    if (CHANNEL) {
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
    {
        constexpr uint32_t TPR = 16 * NQ, RPP = 256 / TPR;
        const uint32_t col = (tid % TPR) * 4, left = j0 + col < vdim ? vdim - j0 - col : 0;
        const float* vb = base + p.v_col + (size_t)a * vdim + j0 + col;
#pragma unroll
        for (uint32_t u = 0; u < kChunk / RPP; ++u) {
            const uint32_t t = tid / TPR + u * RPP;
            *(f32x4_m*)(s_v + t * VW + col) = load4(vb + (size_t)t * p.ld, t < n ? left : 0, aligned);
        }
    }
    __syncthreads();
    if (!out_on) return;
    const uint32_t last = n < pi * 32 + 32 ? n : pi * 32 + 32; // keys up to this half's last row (beyond the chunk's rows: zero scores and values)
    for (uint32_t t0 = 0; t0 < last; t0 += 8)
#pragma unroll
        for (uint32_t u = 0; u < 4; ++u) {
            const uint32_t t = t0 + 2 * u + half;
            const float pa = s_p[row][t];
#pragma unroll
            for (int q = 0; q < NQ; ++q) o[q] = __builtin_amdgcn_mfma_f32_32x32x2f32(pa, s_v[t * VW + pj * 32 * NQ + 32 * q + l32], o[q], 0, 0, 0);
        }
    const float skip = p.skip ? p.skip[a] : 0.0f;
#pragma unroll
    for (int q = 0; q < NQ; ++q) {
        const uint32_t col = pj * 32 * NQ + 32 * q + l32;
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
        const uint32_t vw = p.vdim <= 64 ? 64 : 128, vt = (p.vdim + vw - 1) / vw, kt = (p.dim + 63) / 64;
        const uint32_t aligned = p.ld % 4 == 0 && p.q_col % 4 == 0 && p.k_col % 4 == 0 && p.v_col % 4 == 0 && p.dim % 4 == 0 && p.vdim % 4 == 0 && (uintptr_t)p.rows_in % 16 == 0 &&
                                 (p.per_head || (p.lddecay % 4 == 0 && (uintptr_t)p.decay % 16 == 0)) ? 1u : 0u;
        UZU_REQUIRE((size_t)vt * kt <= 65535 && ((size_t)p.dim * p.vdim + 255) / 256 <= 65535, "decayed_state: head widths %u x %u", p.dim, p.vdim);
        const dim3 lgrid(p.chunks, p.heads, vt * kt), sgrid(p.nseq, p.heads, (uint32_t)(((size_t)p.dim * p.vdim + 255) / 256)), ogrid(p.chunks, p.heads, vt);
        float* ws = p.chunk_ws;
#define UZU_DC(CH, NQ)                                                                                                                                                             \
    do {                                                                                                                                                                           \
        UZU_PROPAGATE(launch_check([&] { hipLaunchKernelGGL((decayed_state_local_kernel<CH, NQ>), lgrid, dim3(256), 0, s, p, ws, aligned); }, "decayed_state_local"));             \
        UZU_PROPAGATE(launch_check([&] { hipLaunchKernelGGL(decayed_state_scan_kernel<CH>, sgrid, dim3(256), 0, s, p, ws); }, "decayed_state_scan"));                              \
        return launch_check([&] { hipLaunchKernelGGL((decayed_state_out_kernel<CH, NQ>), ogrid, dim3(256), 0, s, p, (const float*)ws, aligned); }, "decayed_state_out");           \
    } while (0)
        if (p.per_head) {
            if (vw == 64) UZU_DC(false, 1);
            UZU_DC(false, 2);
        }
        if (vw == 64) UZU_DC(true, 1);
        UZU_DC(true, 2);
#undef UZU_DC
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
