// lm_ssd.hip — the selective state space mixer of the layered-model tier (a scalar decay per head and token, B and C shared by the
// heads of a group) and the row-wise kernels that stand beside it: the norm in equal parts behind its gate, and the polynomial
// activation of a dense feed-forward.  Everything here is fp32 in both precision modes: step sizes, decays and their logarithms,
// the recurrent state, gates, norms.
#include <math.h>
#include <stdlib.h>

#include <algorithm>

#include "lm_kernels.h"

namespace zg {
namespace lm {

namespace {

typedef __attribute__((ext_vector_type(16))) float f32x16_ssd;

__device__ __forceinline__ float silu_f(float z) { return z / (1.0f + expf(-z)); }
__device__ __forceinline__ float softplus_f(float z) { return z > 20.0f ? z : log1pf(expf(z)); }

__device__ __forceinline__ float block_allsum(float v, float* s_red) {
    v = wave_allsum(v);
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, nw = (blockDim.x + 63) >> 6;
    __syncthreads();
    if (lane == 0) s_red[wave] = v;
    __syncthreads();
    float t = 0.0f;
    for (int w = 0; w < nw; ++w) t += s_red[w];
    return t;
}

// ------------------------------------------------------------------------------------------------ token by token
// A workgroup takes an entry, a head and 32 columns of its state [N][V]: thread (row group g, column c) holds R consecutive rows of
// column c, so a state row travels as 128-byte runs.  Tokens are staged kSsdBlock at a time (B and C of the head's group, x of the
// columns, decay and step); the row groups' shares of S^T C meet in the LDS once per block.
// CONV (steps of one row per entry): xbc holds the raw projection columns, and the workgroup convolves the channels it needs over the
// slot's tail itself (the tail is moved on by a later launch, once every workgroup has read it).
constexpr int kSsdCols = 32;
constexpr int kSsdGroups = 8;
constexpr int kSsdBlock = 8;
constexpr int kSsdTaps = 16;
constexpr int kSsdFastTaps = 4;

template <int R, bool CONV>
__global__ __launch_bounds__(256) void ssd_scan_kernel(const SsdArgs a, const ConvArgs cv, const int* ent_start, const int* ent_len, const int* ent_slot) {
    constexpr int Np = R * kSsdGroups;
    constexpr int TB = CONV ? 1 : kSsdBlock;
    __shared__ __attribute__((aligned(16))) float s_B[TB][Np], s_C[TB][Np];
    __shared__ float s_x[TB][kSsdCols], s_part[TB][4][kSsdCols], s_dec[TB], s_dt[TB];
    const int e = blockIdx.x, h = blockIdx.y, tid = threadIdx.x, cl = tid & 31, g = tid >> 5, c = blockIdx.z * kSsdCols + cl;
    const int n = ent_len[e], m0 = ent_start[e], slot = ent_slot[e];
    if (n <= 0) return;
    const bool col_ok = c < a.V;
    const int HV = a.H * a.V, grp = h / (a.H / a.G), oB = HV + grp * a.N, oC = HV + (a.G + grp) * a.N, ox = h * a.V + blockIdx.z * kSsdCols;
    float* Sg = a.state + (size_t)slot * a.slot_stride + (size_t)h * a.N * a.V;
    float S[R];
#pragma unroll
    for (int r = 0; r < R; ++r) {
        const int i = g * R + r;
        S[r] = (col_ok && i < a.N) ? Sg[(size_t)i * a.V + c] : 0.0f;
    }
    const float rate = -expf(a.a_log[h]), bias = a.dt_bias[h], skip = a.skip[h];
    for (int t0 = 0; t0 < n; t0 += TB) {
        const int nb = min(TB, n - t0);
        if (t0 > 0) __syncthreads();  // the block before has been consumed
        for (int idx = tid; idx < nb * (2 * Np + kSsdCols); idx += 256) {
            const int t = idx / (2 * Np + kSsdCols), o = idx % (2 * Np + kSsdCols);
            int ch = -1;  // channel of the row [x | B | C]
            if (o < Np) ch = o < a.N ? oB + o : -1;
            else if (o < 2 * Np) ch = o - Np < a.N ? oC + o - Np : -1;
            else ch = blockIdx.z * kSsdCols + o - 2 * Np < a.V ? ox + o - 2 * Np : -1;
            float v = 0.0f;
            if (ch >= 0) {
                v = a.xbc[(size_t)(m0 + t0 + t) * a.ld_xbc + ch];
                if (CONV) {
                    const float* tl = cv.tail + (size_t)slot * cv.slot_stride;
                    const int K = cv.taps - 1;
                    float acc = cv.bias ? cv.bias[ch] : 0.0f;
                    if (cv.taps <= kSsdFastTaps) {  // weights and tail requested together
                        float wt[kSsdFastTaps], tv[kSsdFastTaps];
#pragma unroll
                        for (int j = 0; j < kSsdFastTaps; ++j) {
                            wt[j] = cv.w[(size_t)ch * cv.taps + min(j, K)];
                            tv[j] = K > 0 ? tl[(size_t)min(j, K - 1) * cv.C + ch] : 0.0f;
                        }
#pragma unroll
                        for (int j = 0; j < kSsdFastTaps; ++j) acc = j <= K ? fmaf(wt[j], j < K ? tv[j] : v, acc) : acc;
                    } else {
                        for (int j = 0; j < cv.taps; ++j) acc = fmaf(cv.w[(size_t)ch * cv.taps + j], j < K ? tl[(size_t)j * cv.C + ch] : v, acc);
                    }
                    v = silu_f(acc);
                }
            }
            if (o < Np) s_B[t][o] = v;
            else if (o < 2 * Np) s_C[t][o - Np] = v;
            else s_x[t][o - 2 * Np] = v;
        }
        if (tid < nb) {
            const float dt = softplus_f(a.dt[(size_t)(m0 + t0 + tid) * a.ld_proj + h] + bias);
            s_dt[tid] = dt;
            s_dec[tid] = expf(rate * dt);
        }
        __syncthreads();
        for (int t = 0; t < nb; ++t) {
            const float dec = s_dec[t], xv = s_x[t][cl] * s_dt[t];
            float o = 0.0f;
#pragma unroll
            for (int r = 0; r < R; ++r) {
                S[r] = fmaf(dec, S[r], s_B[t][g * R + r] * xv);
                o = fmaf(S[r], s_C[t][g * R + r], o);
            }
            o += __shfl_xor(o, 32, 64);
            if ((tid & 63) < 32) s_part[t][tid >> 6][cl] = o;
        }
        __syncthreads();
        for (int idx = tid; idx < nb * kSsdCols; idx += 256) {
            const int t = idx / kSsdCols, cc = idx % kSsdCols, col = blockIdx.z * kSsdCols + cc;
            if (col < a.V) {
                const float y = (s_part[t][0][cc] + s_part[t][1][cc]) + (s_part[t][2][cc] + s_part[t][3][cc]) + skip * s_x[t][cc];
                const size_t m = m0 + t0 + t;
                a.out[m * a.ldo + (size_t)h * a.V + col] = y * silu_f(a.z[m * a.ld_proj + (size_t)h * a.V + col]);
            }
        }
    }
#pragma unroll
    for (int r = 0; r < R; ++r) {
        const int i = g * R + r;
        if (col_ok && i < a.N) Sg[(size_t)i * a.V + c] = S[r];
    }
}

// ------------------------------------------------------------------------------------------------ chunks on the matrix cores
// With one decay per head and token the recurrence of a chunk of n <= 32 tokens is three matrix products (true fp32,
// v_mfma_f32_32x32x2_f32); l_t = -exp(a_log) dt_t, L(j, i) = exp(l_(j+1) + ... + l_i):
//   state   E = sum_j L(j, n-1) dt_j B_j x_j^T                      the chunk's end state from zero          (per chunk)
//   carry   S_start(c + 1) = L(-1, n-1) S_start(c) + E_c            down the chunks of an entry              (launch_state_carry)
//   output  y_i = sum_(j<=i) L(j, i) dt_j (C_i . B_j) x_j + L(-1, i) S_start^T C_i + skip x_i, times silu(z)  (per chunk; the skip
//           factor rides on the diagonal of the first sum's weights)
// The logarithms inside a chunk are added up directly between j and i (all of one sign: nothing cancels, and a token that forgets
// everything does not blur the decays behind it).
constexpr int kSsdChunk = 32;

__device__ __forceinline__ bool ssd_find_chunk(int id, const int* ent_len, int n_entries, int& e, int& c) {
    for (e = 0; e < n_entries; ++e) {
        const int nc = (ent_len[e] + kSsdChunk - 1) / kSsdChunk;
        if (id < nc) {
            c = id;
            return true;
        }
        id -= nc;
    }
    return false;
}

__global__ __launch_bounds__(256) void ssd_chunk_state_kernel(const SsdArgs a, const int* ent_start, const int* ent_len, int n_entries,
                                                              float* __restrict__ wsB, float* __restrict__ wsA) {
    __shared__ float s_l[kSsdChunk], s_w[kSsdChunk];
    int e, c;
    if (!ssd_find_chunk(blockIdx.x, ent_len, n_entries, e, c)) return;
    const int h = blockIdx.y, lane = threadIdx.x & 63, wave = threadIdx.x >> 6, r = lane & 31, kh = lane >> 5;
    const int n = min(kSsdChunk, ent_len[e] - c * kSsdChunk), m0 = ent_start[e] + c * kSsdChunk;
    const int HV = a.H * a.V, grp = h / (a.H / a.G);
    const float* base = a.xbc + (size_t)m0 * a.ld_xbc;
    float* E = wsB + ((size_t)blockIdx.x * a.H + h) * a.N * a.V;
    const int tilesN = (a.N + 31) / 32, tilesV = (a.V + 31) / 32;
    float av[16], bv[16];
    auto fetch = [&](int tile) {  // the token is the inner dimension (tokens beyond the chunk's end weigh nothing)
        const int ob = HV + grp * a.N + min((tile / tilesV) * 32 + r, a.N - 1), ox = h * a.V + min((tile % tilesV) * 32 + r, a.V - 1);
#pragma unroll
        for (int t = 0; t < 16; ++t) {
            const float* row = base + min(kh * 16 + t, n - 1) * a.ld_xbc;
            av[t] = row[ob];
            bv[t] = row[ox];
        }
    };
    int tile = blockIdx.z * 4 + wave;
    if (tile < tilesN * tilesV) fetch(tile);  // in flight beside the step sizes
    float dt = 0.0f;
    if (threadIdx.x < kSsdChunk) {
        const int t = threadIdx.x;
        if (t < n) dt = softplus_f(a.dt[(size_t)(m0 + t) * a.ld_proj + h] + a.dt_bias[h]);
        s_l[t] = -expf(a.a_log[h]) * dt;
    }
    __syncthreads();
    if (threadIdx.x < kSsdChunk) {  // (tokens beyond the chunk's end: dt = 0, l = 0)
        float run = 0.0f;
        for (int t = kSsdChunk - 1; t > (int)threadIdx.x; --t) run += s_l[t];
        s_w[threadIdx.x] = dt * expf(run);
        if (threadIdx.x == 0 && blockIdx.z == 0) wsA[(size_t)blockIdx.x * a.H + h] = expf(run + s_l[0]);
    }
    __syncthreads();
    for (bool first = true; tile < tilesN * tilesV; tile += 4 * gridDim.z, first = false) {
        const int i0 = (tile / tilesV) * 32, v0 = (tile % tilesV) * 32;
        if (!first) fetch(tile);
        f32x16_ssd acc;
#pragma unroll
        for (int i = 0; i < 16; ++i) acc[i] = 0.0f;
#pragma unroll
        for (int t = 0; t < 16; ++t) acc = __builtin_amdgcn_mfma_f32_32x32x2f32(av[t] * s_w[kh * 16 + t], bv[t], acc, 0, 0, 0);
        // accumulator element i: row 8 (i / 4) + 4 half + i % 4, column r
#pragma unroll
        for (int i = 0; i < 16; ++i) {
            const int row = i0 + 8 * (i >> 2) + 4 * kh + (i & 3);
            if (row < a.N && v0 + r < a.V) E[(size_t)row * a.V + v0 + r] = acc[i];
        }
    }
}

// A workgroup takes a chunk and up to `hb` heads of one group.  The products C_i . B_j are the group's: the four waves split the
// state channels (eight at a time), their shares meet in the LDS; then a wave owns (head, 32 value columns) units.
constexpr int kSsdHeads = 4;  // most heads of a workgroup

__global__ __launch_bounds__(256, 2) void ssd_chunk_out_kernel(const SsdArgs a, const int* ent_start, const int* ent_len, int n_entries,
                                                            const float* __restrict__ wsB, int hb, int blocks_per_group) {
    extern __shared__ __attribute__((aligned(16))) float s_ssd[];
    __shared__ float s_p[4][32][33];
    __shared__ float s_l[kSsdHeads][32], s_dt[kSsdHeads][32], s_pre[kSsdHeads][32];
    int e, c;
    if (!ssd_find_chunk(blockIdx.x, ent_len, n_entries, e, c)) return;
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, r = lane & 31, kh = lane >> 5;
    const int n = min(kSsdChunk, ent_len[e] - c * kSsdChunk), m0 = ent_start[e] + c * kSsdChunk;
    const int grp = blockIdx.y / blocks_per_group, per = a.H / a.G;
    const int hl0 = (blockIdx.y % blocks_per_group) * hb, nh = min(hb, per - hl0), h0 = grp * per + hl0;  // heads [h0, h0 + nh)
    const int HV = a.H * a.V, N8 = (a.N + 31) / 32 * 4, ldC = 8 * N8 + 4;  // (groups of eight state channels, a multiple of four of them)
    float* s_C = s_ssd;  // [32][ldC], zero beyond N (rows beyond the chunk repeat its last one: nothing of them is written)
    const float* brow = a.xbc + (size_t)m0 * a.ld_xbc + HV + (size_t)grp * a.N;
    const float* crow = brow + (size_t)a.G * a.N;
    const bool vec = a.N % 4 == 0 && a.ld_xbc % 4 == 0 && HV % 4 == 0 && (reinterpret_cast<uintptr_t>(a.xbc) & 15) == 0;
    // four channels of a row; beyond N whatever is there (the query rows hold zeros beyond N, so it weighs nothing)
    auto row4 = [&](const float* row, int ch) {
        if (vec) return *reinterpret_cast<const f32x4*>(row + min(ch, a.N - 4));
        return f32x4{row[min(ch, a.N - 1)], row[min(ch + 1, a.N - 1)], row[min(ch + 2, a.N - 1)], row[min(ch + 3, a.N - 1)]};
    };
    {
        const int t = tid >> 3;
        for (int ch = 4 * (tid & 7); ch < 8 * N8; ch += 32) {
            f32x4 v = row4(crow + (size_t)min(t, n - 1) * a.ld_xbc, ch);
            v.x = ch + 0 < a.N ? v.x : 0.0f;
            v.y = ch + 1 < a.N ? v.y : 0.0f;
            v.z = ch + 2 < a.N ? v.z : 0.0f;
            v.w = ch + 3 < a.N ? v.w : 0.0f;
            *reinterpret_cast<f32x4*>(s_C + t * ldC + ch) = v;
        }
    }
    if (tid < 32 * nh) {
        const int hh = tid >> 5, t = tid & 31;
        const float dt = t < n ? softplus_f(a.dt[(size_t)(m0 + t) * a.ld_proj + h0 + hh] + a.dt_bias[h0 + hh]) : 0.0f;
        s_dt[hh][t] = dt;
        s_l[hh][t] = -expf(a.a_log[h0 + hh]) * dt;
    }
    __syncthreads();
    if (tid < 32 * nh) {
        const int hh = tid >> 5, t = tid & 31;
        float run = 0.0f;
        for (int u = 0; u <= t; ++u) run += s_l[hh][u];
        s_pre[hh][t] = expf(run);  // what the start state has decayed to when token t reads it
    }
    f32x16_ssd acc;
#pragma unroll
    for (int i = 0; i < 16; ++i) acc[i] = 0.0f;
    {
        const float* br = brow + (size_t)min(r, n - 1) * a.ld_xbc;
        // channels 8 g8 + 4 half + u of rows r: query row from the LDS, key row from memory (requested one group ahead)
        f32x4 kn = row4(br, 8 * wave + 4 * kh);
        for (int g8 = wave; g8 < N8; g8 += 4) {
            const f32x4 k = kn, q = *reinterpret_cast<const f32x4*>(s_C + r * ldC + 8 * g8 + 4 * kh);
            kn = row4(br, 8 * (g8 + 4) + 4 * kh);
            acc = __builtin_amdgcn_mfma_f32_32x32x2f32(q.x, k.x, acc, 0, 0, 0);
            acc = __builtin_amdgcn_mfma_f32_32x32x2f32(q.y, k.y, acc, 0, 0, 0);
            acc = __builtin_amdgcn_mfma_f32_32x32x2f32(q.z, k.z, acc, 0, 0, 0);
            acc = __builtin_amdgcn_mfma_f32_32x32x2f32(q.w, k.w, acc, 0, 0, 0);
        }
#pragma unroll
        for (int i = 0; i < 16; ++i) s_p[wave][8 * (i >> 2) + 4 * kh + (i & 3)][r] = acc[i];
    }
    __syncthreads();
    for (int idx = tid; idx < 1024; idx += 256) {  // the waves' shares, in a fixed order
        const int i = idx >> 5, j = idx & 31;
        s_p[0][i][j] = (s_p[0][i][j] + s_p[1][i][j]) + (s_p[2][i][j] + s_p[3][i][j]);
    }
    __syncthreads();
    const int tilesV = (a.V + 31) / 32;
    for (int u = wave; u < nh * tilesV; u += 4) {
        const int hh = u / tilesV, h = h0 + hh, v0 = (u % tilesV) * 32;
        const bool col_ok = v0 + r < a.V;
        // (columns beyond V read the last one, tokens beyond the chunk its last: they weigh nothing or are not written)
        const int col = h * a.V + min(v0 + r, a.V - 1);
        const float* xbase = a.xbc + (size_t)m0 * a.ld_xbc + col;
        const float* S = wsB + (size_t)blockIdx.x * a.H * a.N * a.V + (size_t)h * a.N * a.V + min(v0 + r, a.V - 1);  // the chunk's start state (the carry left it here)
        float xv[16];
#pragma unroll
        for (int t = 0; t < 16; ++t) xv[t] = xbase[min(kh * 16 + t, n - 1) * a.ld_xbc];
        float* obase = a.out + (size_t)m0 * a.ldo + col;
        const float* zbase = a.z + (size_t)m0 * a.ld_proj + col;
        float zv[16];  // the gates of the outputs this lane will write
#pragma unroll
        for (int i = 0; i < 16; ++i) {
            const int qi = 8 * (i >> 2) + 4 * kh + (i & 3);
            zv[i] = zbase[min(qi, n - 1) * a.ld_proj];
        }
        // the start state's share, 16 state rows requested while the 16 before are multiplied
        f32x16_ssd accS;
#pragma unroll
        for (int i = 0; i < 16; ++i) {
            acc[i] = 0.0f;
            accS[i] = 0.0f;
        }
        float sv[2][8];
        auto state_rows = [&](int g0, float* dst) {
#pragma unroll
            for (int t = 0; t < 8; ++t) {
                const int ch = 8 * (g0 + (t >> 2)) + 4 * kh + (t & 3);
                dst[t] = S[min(ch, a.N - 1) * a.V];
            }
        };
        auto state_product = [&](int g0, const float* src) {
#pragma unroll
            for (int t4 = 0; t4 < 2; ++t4) {
                const f32x4 q = *reinterpret_cast<const f32x4*>(s_C + r * ldC + 8 * (g0 + t4) + 4 * kh);
                accS = __builtin_amdgcn_mfma_f32_32x32x2f32(q.x, src[4 * t4 + 0], accS, 0, 0, 0);
                accS = __builtin_amdgcn_mfma_f32_32x32x2f32(q.y, src[4 * t4 + 1], accS, 0, 0, 0);
                accS = __builtin_amdgcn_mfma_f32_32x32x2f32(q.z, src[4 * t4 + 2], accS, 0, 0, 0);
                accS = __builtin_amdgcn_mfma_f32_32x32x2f32(q.w, src[4 * t4 + 3], accS, 0, 0, 0);
            }
        };
        state_rows(0, sv[0]);
        for (int g0 = 0; g0 < N8; g0 += 4) {
            state_rows(g0 + 2, sv[1]);
            state_product(g0, sv[0]);
            if (g0 + 4 < N8) state_rows(g0 + 4, sv[0]);
            state_product(g0 + 2, sv[1]);
        }
        // the chunk's own tokens: lane (r, half) weighs the keys half * 16 .. + 15 for query row r, from the nearest back
        float wv[16], run = 0.0f;
        const float skip = a.skip[h];
        if (kh == 0)
            for (int t = 16; t < 32; ++t) run += t <= r ? s_l[hh][t] : 0.0f;
#pragma unroll
        for (int t = 15; t >= 0; --t) {
            const int j = kh * 16 + t;
            if (t < 15 && j < r) run += s_l[hh][j + 1];
            if (t == 15 && kh == 1) run = 0.0f;
            wv[t] = j <= r ? s_p[0][r][j] * expf(run) * s_dt[hh][j] + (j == r ? skip : 0.0f) : 0.0f;
        }
#pragma unroll
        for (int t = 0; t < 16; ++t) acc = __builtin_amdgcn_mfma_f32_32x32x2f32(wv[t], xv[t], acc, 0, 0, 0);
#pragma unroll
        for (int i = 0; i < 16; ++i) {
            const int qi = 8 * (i >> 2) + 4 * kh + (i & 3);
            if (qi < n && col_ok) obase[qi * a.ldo] = (acc[i] + s_pre[hh][qi] * accS[i]) * silu_f(zv[i]);
        }
    }
}

// ------------------------------------------------------------------------------------------------ norm in parts, polynomial activation
constexpr int kPartRegs = 16;  // parts of up to 256 * kPartRegs channels stay in registers

__global__ __launch_bounds__(256) void part_norm_kernel(float* v, int ld, int width, int parts, const float* w, float eps, const ConvArgs cv, const int* row_slot) {
    __shared__ float s_red[8];
    const int m = blockIdx.x, part = blockIdx.y, n = width / parts;
    if (part >= parts) {  // the row is its entry's only one: the workgroups behind the parts move the convolution's tail on, 256 channels each
        const int K = cv.taps - 1, c = (part - parts) * 256 + threadIdx.x;
        if (c >= cv.C) return;
        float* tl = cv.tail + (size_t)row_slot[m] * cv.slot_stride + c;
        float val = cv.in[(size_t)m * cv.ld_in + c];  // every entry takes its successor's place, the newest one the current input
        for (int i = K - 1; i >= 0; --i) {
            const float old = tl[(size_t)i * cv.C];
            tl[(size_t)i * cv.C] = val;
            val = old;
        }
        return;
    }
    float* p = v + (size_t)m * ld + (size_t)part * n;
    const float* wp = w + (size_t)part * n;
    if (n <= 256 * kPartRegs) {
        float x[kPartRegs], wr[kPartRegs], ss = 0.0f;
#pragma unroll
        for (int j = 0; j < kPartRegs; ++j) {
            const int i = threadIdx.x + 256 * j;
            x[j] = i < n ? p[i] : 0.0f;
            wr[j] = i < n ? wp[i] : 0.0f;
            ss = fmaf(x[j], x[j], ss);
        }
        ss = block_allsum(ss, s_red);
        const float rn = 1.0f / sqrtf(ss / (float)n + eps);
#pragma unroll
        for (int j = 0; j < kPartRegs; ++j) {
            const int i = threadIdx.x + 256 * j;
            if (i < n) p[i] = x[j] * rn * wr[j];
        }
        return;
    }
    float ss = 0.0f;
    for (int i = threadIdx.x; i < n; i += 256) ss = fmaf(p[i], p[i], ss);
    ss = block_allsum(ss, s_red);
    const float rn = 1.0f / sqrtf(ss / (float)n + eps);
    for (int i = threadIdx.x; i < n; i += 256) p[i] = p[i] * rn * wp[i];
}

__global__ __launch_bounds__(256) void polynorm_kernel(float* z, int ld, int F, const float* act, float eps) {
    __shared__ float s_red[3][4];
    float* p = z + (size_t)blockIdx.x * ld;
    const float ca = act[0], cb = act[1], cc = act[2], ce = act[3];
    float x[kPartRegs], s1 = 0.0f, s2 = 0.0f, s3 = 0.0f;
    const bool held = F <= 256 * kPartRegs;
    if (held) {
#pragma unroll
        for (int j = 0; j < kPartRegs; ++j) {
            const int i = threadIdx.x + 256 * j;
            x[j] = i < F ? p[i] : 0.0f;
        }
#pragma unroll
        for (int j = 0; j < kPartRegs; ++j) {
            const float q = x[j] * x[j], q2 = q * q;
            s1 += q;
            s2 += q2;
            s3 = fmaf(q2, q, s3);
        }
    } else {
        for (int i = threadIdx.x; i < F; i += 256) {
            const float q = p[i] * p[i], q2 = q * q;
            s1 += q;
            s2 += q2;
            s3 = fmaf(q2, q, s3);
        }
    }
    s1 = wave_allsum(s1);
    s2 = wave_allsum(s2);
    s3 = wave_allsum(s3);
    if ((threadIdx.x & 63) == 0) {
        const int w = threadIdx.x >> 6;
        s_red[0][w] = s1;
        s_red[1][w] = s2;
        s_red[2][w] = s3;
    }
    __syncthreads();
    auto inv = [&](int k) { return 1.0f / sqrtf(((s_red[k][0] + s_red[k][1]) + (s_red[k][2] + s_red[k][3])) / (float)F + eps); };
    const float f1 = ca * inv(0), f2 = cb * inv(1), f3 = cc * inv(2);
    if (held) {
#pragma unroll
        for (int j = 0; j < kPartRegs; ++j) {
            const int i = threadIdx.x + 256 * j;
            if (i < F) p[i] = fmaf(fmaf(fmaf(f3, x[j], f2), x[j], f1), x[j], ce);
        }
    } else {
        for (int i = threadIdx.x; i < F; i += 256) p[i] = fmaf(fmaf(fmaf(f3, p[i], f2), p[i], f1), p[i], ce);
    }
}

}  // namespace

size_t ssd_workspace(int M, int n_entries, int H, int N, int V) {
    const size_t chunks = (size_t)(M + kSsdChunk - 1) / kSsdChunk + n_entries;
    return chunks * ((size_t)H * N * V + H);
}

int launch_ssd_scan(const SsdArgs& a, const ConvArgs* conv, int M, const int* ent_start, const int* ent_len, const int* ent_slot, int n_entries,
                    float* ws, size_t ws_floats, hipStream_t s) {
    if (n_entries <= 0 || M <= 0) return ZG_OK;
    ZG_REQUIRE(a.H >= 1 && a.G >= 1 && a.H % a.G == 0 && a.N >= 1 && a.N <= kSsdMaxState && a.V >= 1 && a.H <= 65535, ZG_ERR_UNSUPPORTED,
               "state space: %d heads in %d groups, a state of %d x %d per head (at most %d rows)", a.H, a.G, a.N, a.V, kSsdMaxState);
    ZG_REQUIRE(!conv || (M == n_entries && conv->taps >= 1 && conv->taps <= kSsdTaps && conv->C == a.H * a.V + 2 * a.G * a.N), ZG_ERR_ARG,
               "state space: the convolution inside the scan is for one row per entry and at most %d taps", kSsdTaps);
    const int n_chunks = (M + kSsdChunk - 1) / kSsdChunk + n_entries;
    if (!conv && M > kGemvMaxRows && ws && ws_floats >= ssd_workspace(M, n_entries, a.H, a.N, a.V) && getenv("ZGPT2_LM_SSD_NO_CHUNKS") == nullptr) {
        // prompt portions: chunks of kSsdChunk tokens as matrix products (the test hook sends them through the scan)
        float* cB = ws;
        float* cA = ws + (size_t)n_chunks * a.H * a.N * a.V;
        const int tiles = ((a.N + 31) / 32) * ((a.V + 31) / 32);
        ssd_chunk_state_kernel<<<dim3(n_chunks, a.H, std::min(16, (tiles + 3) / 4)), 256, 0, s>>>(a, ent_start, ent_len, n_entries, cB, cA);
        ZG_HIP(hipGetLastError());
        ZG_TRY(launch_state_carry(a.state, a.slot_stride, ent_len, ent_slot, n_entries, a.H, a.N, a.V, cB, cA, 1, kSsdChunk, s));
        const int tilesV = (a.V + 31) / 32, per = a.H / a.G, hb = std::max(1, std::min(std::min(kSsdHeads, per), 4 / tilesV)), bpg = (per + hb - 1) / hb;
        const size_t lds = (size_t)32 * ((a.N + 31) / 32 * 32 + 4) * sizeof(float);
        ssd_chunk_out_kernel<<<dim3(n_chunks, a.G * bpg), 256, lds, s>>>(a, ent_start, ent_len, n_entries, cB, hb, bpg);
        ZG_HIP(hipGetLastError());
        return ZG_OK;
    }
    const ConvArgs cv = conv ? *conv : ConvArgs();
    const int rr = (a.N + kSsdGroups - 1) / kSsdGroups;
    const dim3 grid(n_entries, a.H, (a.V + kSsdCols - 1) / kSsdCols);
#define ZG_SSD(R_)                                                                                       \
    do {                                                                                                 \
        if (conv) ssd_scan_kernel<R_, true><<<grid, 256, 0, s>>>(a, cv, ent_start, ent_len, ent_slot);   \
        else ssd_scan_kernel<R_, false><<<grid, 256, 0, s>>>(a, cv, ent_start, ent_len, ent_slot);       \
    } while (0)
    if (rr <= 2) ZG_SSD(2);
    else if (rr <= 4) ZG_SSD(4);
    else if (rr <= 8) ZG_SSD(8);
    else if (rr <= 16) ZG_SSD(16);
    else ZG_SSD(32);
#undef ZG_SSD
    ZG_HIP(hipGetLastError());
    return ZG_OK;
}

int launch_part_norm(float* v, int ld, int width, int parts, int M, const float* w, float eps, const ConvArgs* conv, const int* row_slot, hipStream_t s) {
    if (M <= 0 || width <= 0) return ZG_OK;
    ZG_REQUIRE(parts >= 1 && parts <= 65535 && width % parts == 0, ZG_ERR_ARG, "norm in parts: %d channels in %d parts", width, parts);
    ZG_REQUIRE(!conv || (conv->taps >= 1 && conv->taps <= kSsdTaps), ZG_ERR_ARG, "norm in parts: a convolution of more than %d taps", kSsdTaps);
    const int tail_blocks = conv && conv->taps > 1 ? (conv->C + 255) / 256 : 0;
    part_norm_kernel<<<dim3(M, parts + tail_blocks), 256, 0, s>>>(v, ld, width, parts, w, eps, conv ? *conv : ConvArgs(), row_slot);
    ZG_HIP(hipGetLastError());
    return ZG_OK;
}

int launch_polynorm(float* z, int ld, int F, int M, const float* act, float eps, hipStream_t s) {
    if (M <= 0 || F <= 0) return ZG_OK;
    polynorm_kernel<<<M, 256, 0, s>>>(z, ld, F, act, eps);
    ZG_HIP(hipGetLastError());
    return ZG_OK;
}

}  // namespace lm
}  // namespace zg
