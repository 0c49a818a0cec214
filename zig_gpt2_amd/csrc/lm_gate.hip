// lm_gate.hip — attention whose weights are sigmoids: a visible key weighs sigmoid(scale q . k + bias[h]) and nothing is normalised over
// the keys.  A row's result is a plain sum, so shares of its keys add up in any grouping and no pass over the scores is needed in
// front of the values:
//   * gate_rows_kernel    steps of few rows (decode): a workgroup of sixteen waves per (share of the keys, row, key head), eight keys to a
//                         wave and trip, up to four query heads of the key head on every key read (one, while there are few rows and heads:
//                         a compute unit is then busy with the weights and sums of its heads, not with its loads).  Steps of one row per entry
//                         also prepare the row here — rotary q and k, the value's norm and mix, the token's cache row.
//   * gate_tiles_kernel   prompt portions: 32 consecutive rows of an entry and one head per workgroup, tiles of 32 keys dealt to the four
//                         waves; both products on the matrix cores, operands straight from the cache rows to registers.
#include <math.h>
#include <stdlib.h>

#include <algorithm>

#include "lm_kernels.h"

namespace zg {
namespace lm {

namespace {

typedef __attribute__((ext_vector_type(8))) __bf16 bf16x8;
typedef __attribute__((ext_vector_type(16))) float f32x16;

__device__ __forceinline__ float sigmoid_f(float z) { return 1.0f / (1.0f + expf(-z)); }

__device__ __forceinline__ int first_key(int pos, const KeyMask& mask) {
    return mask.chunk > 0 ? pos - pos % mask.chunk : mask.window > 0 ? max(0, pos - mask.window + 1) : 0;
}
__device__ __forceinline__ int cache_row(const int* pages, int j, int page_tokens, int max_pages) {
    return pages[(j / page_tokens) % max_pages] * page_tokens + j % page_tokens;
}

struct GateArgs {
    const float* q;
    int ldq;
    float* out;
    int ldo;
    int H, G, D, V;
    float scale;
    const float* bias;  // [H]
    KeyMask mask;
    const int *row_pos, *row_slot, *page_table;
    int max_pages, page_tokens;
    float* cache;
};

// ------------------------------------------------------------------------------------------------ few rows
constexpr int kGateWaves = 16;
constexpr int kGateKeys = 8;   // keys of a wave per trip: eight lanes share a key's channels

// channel i of a vector of rot.dims turned channels at position pos
__device__ __forceinline__ float rotary_at(const float* v, int i, float fpos, const Rotary& rot) {
    if (i >= rot.dims) return v[i];
    const int half = rot.dims / 2;
    const bool second = rot.halves ? i >= half : (i & 1);
    float sn, cs;
    sincosf(fpos * rot.freq[rot.halves ? (second ? i - half : i) : i >> 1], &sn, &cs);
    const float own = v[i], other = v[rot.halves ? (second ? i - half : i + half) : i ^ 1];
    return (second ? own * cs + other * sn : own * cs - other * sn) * rot.amp;
}

// KC: 8 KC >= D (channels of a key a lane holds); VC: 64 VC >= V; U: trips whose rows are requested together; NH: query heads of one
// key head per workgroup.
// PREP: the row's q is rotated on its way in; its own key and value are prepared here, filed in the cache and used from the LDS by the
// workgroup whose share ends with them.
template <int KC, int VC, int U, int NH, bool PREP>
__global__ __launch_bounds__(64 * kGateWaves) void gate_rows_kernel(const GateArgs a, const Rotary rot, const ValuePrep vals, float* po) {
    constexpr int DP = 8 * KC, VP = 64 * VC;
    __shared__ __attribute__((aligned(16))) float s_q[NH * DP];
    __shared__ __attribute__((aligned(16))) float s_own[DP + VP];
    __shared__ float s_o[kGateWaves][NH][VP];
    const int split = blockIdx.x, n_split = gridDim.x, m = blockIdx.y, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const int rep = a.H / a.G, hchunks = (rep + NH - 1) / NH, g = blockIdx.z / hchunks, hc = blockIdx.z % hchunks;
    const int h0 = g * rep + hc * NH, nh = min(NH, rep - hc * NH);
    const int D = a.D, V = a.V, pos = a.row_pos[m];
    const int* pages = a.page_table + (size_t)a.row_slot[m] * a.max_pages;
    const size_t cstride = (size_t)a.G * (D + V);
    const int k_first = first_key(pos, a.mask), n_keys = pos - k_first + 1;
    const int share = (n_keys + n_split - 1) / n_split;
    const int k_lo = k_first + min(n_keys, split * share), k_hi = k_first + min(n_keys, (split + 1) * share);
    const bool owns = PREP && k_hi == pos + 1 && k_lo < k_hi;  // this share ends with the row's own key
    const float* row = a.q + (size_t)m * a.ldq;
    const int l8 = lane & 7, kk = lane >> 3;  // the lane's channels and key of a trip
    const bool vec = D % 4 == 0 && V % 4 == 0 && (reinterpret_cast<uintptr_t>(a.cache) & 15) == 0;

    const int k_end = owns ? k_hi - 1 : k_hi;  // keys that the cache holds
    // U trips' rows at once; the first ones are on their way while q is staged
    float kr[U][KC], vr[U][kGateKeys][VC];
    auto fetch = [&](int t0) {
        int crow[U];
#pragma unroll
        for (int u = 0; u < U; ++u) {
            crow[u] = cache_row(pages, min(t0 + u * kGateWaves * kGateKeys + kk, k_end - 1), a.page_tokens, a.max_pages);
        }
#pragma unroll
        for (int u = 0; u < U; ++u) {
            const float* kp = a.cache + (size_t)crow[u] * cstride + (size_t)g * D;
            if (vec) {
#pragma unroll
                for (int i = 0; i < KC; i += 4) {
                    const int d = 8 * i + 4 * l8;  // eight lanes read 128 consecutive bytes
                    const f32x4 x = *reinterpret_cast<const f32x4*>(kp + (d < D ? d : 0));  // (q is zero beyond D)
                    kr[u][i] = x.x; kr[u][i + 1] = x.y; kr[u][i + 2] = x.z; kr[u][i + 3] = x.w;
                }
            } else {
#pragma unroll
                for (int i = 0; i < KC; ++i) {
                    const int d = 8 * (i & ~3) + 4 * l8 + (i & 3);
                    kr[u][i] = kp[min(d, D - 1)];
                }
            }
#pragma unroll
            for (int e = 0; e < kGateKeys; ++e) {
                const int rw = __builtin_amdgcn_readlane(crow[u], 8 * e);
                const float* vp = a.cache + (size_t)rw * cstride + (size_t)a.G * D + (size_t)g * V;
#pragma unroll
                for (int c = 0; c < VC; ++c) vr[u][e][c] = vp[min(lane + 64 * c, V - 1)];
            }
        }
    };
    const int t_first = k_lo + wave * kGateKeys;
    if (t_first < k_end) fetch(t_first);

    for (int i = tid; i < NH * DP; i += blockDim.x) {
        const int hh = i / DP, d = i % DP;
        float v = 0.0f;
        if (hh < nh && d < D) {
            const float* qh = row + (size_t)(h0 + hh) * D;
            v = PREP ? rotary_at(qh, d, (float)pos, rot) : qh[d];
        }
        s_q[i] = v;
    }
    if (owns) {
        float* crow = a.cache + (size_t)cache_row(pages, pos, a.page_tokens, a.max_pages) * cstride;
        const bool files = hc == 0;  // (the other workgroups of the key head prepare the same values for themselves)
        const float* k = row + (size_t)a.H * D + (size_t)g * D;
        for (int i = tid; i < DP; i += blockDim.x) {
            const float v = i < D ? rotary_at(k, i, (float)pos, rot) : 0.0f;
            s_own[i] = v;
            if (files && i < D) crow[(size_t)g * D + i] = v;
        }
        if (wave == kGateWaves - 1) {
            const float* v = row + (size_t)a.H * D + (size_t)a.G * D + (size_t)g * V;
            float r = 1.0f;
            if (vals.norm) {
                float ss = 0.0f;
                for (int i = lane; i < V; i += 64) ss = fmaf(v[i], v[i], ss);
                r = 1.0f / sqrtf(wave_allsum(ss) / (float)V + vals.eps);
            }
            const float lam = vals.mix_first ? *vals.lam : 0.0f;
            for (int i = lane; i < VP; i += 64) {
                float x = 0.0f;
                if (i < V) {
                    const size_t at = ((size_t)m * a.G + g) * V + i;
                    x = v[i] * r;
                    if (vals.first_out && files) vals.first_out[at] = x;
                    if (vals.mix_first) x = fmaf(lam, vals.mix_first[at], (1.0f - lam) * x);
                    if (files) crow[(size_t)a.G * D + (size_t)g * V + i] = x;
                }
                s_own[DP + i] = x;
            }
        }
    }
    float acc[NH][VC];
#pragma unroll
    for (int h = 0; h < NH; ++h)
#pragma unroll
        for (int c = 0; c < VC; ++c) acc[h][c] = 0.0f;
    float hb[NH];
#pragma unroll
    for (int h = 0; h < NH; ++h) hb[h] = h < nh ? a.bias[h0 + h] : 0.0f;
    __syncthreads();

    for (int t0 = t_first; t0 < k_end; t0 += U * kGateWaves * kGateKeys) {
        if (t0 != t_first) fetch(t0);
#pragma unroll
        for (int u = 0; u < U; ++u) {
            const int j = t0 + u * kGateWaves * kGateKeys + kk;
#pragma unroll
            for (int h = 0; h < NH; ++h) {
                float sc = 0.0f;
#pragma unroll
                for (int i = 0; i < KC; ++i) sc = fmaf(s_q[h * DP + 8 * (i & ~3) + 4 * l8 + (i & 3)], kr[u][i], sc);
                sc += __shfl_xor(sc, 1, 64);
                sc += __shfl_xor(sc, 2, 64);
                sc += __shfl_xor(sc, 4, 64);
                const float w = j < k_end ? sigmoid_f(fmaf(sc, a.scale, hb[h])) : 0.0f;
#pragma unroll
                for (int e = 0; e < kGateKeys; ++e) {
                    const float we = __builtin_bit_cast(float, __builtin_amdgcn_readlane(__builtin_bit_cast(int, w), 8 * e));
#pragma unroll
                    for (int c = 0; c < VC; ++c) acc[h][c] = fmaf(we, vr[u][e][c], acc[h][c]);
                }
                __builtin_amdgcn_sched_barrier(0);  // (the heads' q would all be fetched together and not fit the registers)
            }
        }
    }
    if (owns && wave == 0) {
#pragma unroll
        for (int h = 0; h < NH; ++h) {
            float sc = 0.0f;
            for (int d = lane; d < DP; d += 64) sc = fmaf(s_q[h * DP + d], s_own[d], sc);
            const float w = sigmoid_f(fmaf(wave_allsum(sc), a.scale, hb[h]));
#pragma unroll
            for (int c = 0; c < VC; ++c) acc[h][c] = fmaf(w, s_own[DP + lane + 64 * c], acc[h][c]);
        }
    }
#pragma unroll
    for (int h = 0; h < NH; ++h)
#pragma unroll
        for (int c = 0; c < VC; ++c) s_o[wave][h][lane + 64 * c] = acc[h][c];
    __syncthreads();
    float* o = n_split > 1 ? po + ((size_t)m * n_split + split) * a.H * V : a.out + (size_t)m * a.ldo;
    for (int i = tid; i < nh * V; i += blockDim.x) {
        const int h = i / V, c = i % V;
        float t = 0.0f;
#pragma unroll
        for (int w = 0; w < kGateWaves; ++w) t += s_o[w][h][c];
        o[(size_t)(h0 + h) * V + c] = t;
    }
}

// the shares of a row added in order
__global__ __launch_bounds__(256) void gate_merge_kernel(const float* po, int n_split, float* out, int ldo, int HV) {
    const int m = blockIdx.x, o = blockIdx.y * 256 + threadIdx.x;
    if (o >= HV) return;
    const float* base = po + (size_t)m * n_split * HV + o;
    float t = 0.0f;
#pragma unroll 8
    for (int s = 0; s < n_split; ++s) t += base[(size_t)s * HV];
    out[(size_t)m * ldo + o] = t;
}

// ------------------------------------------------------------------------------------------------ prompt portions
// Both products are computed transposed (S^T = K Q^T, O^T = V^T P^T): a lane's column is a query row, and the sixteen weights a lane
// computes — keys 8 (i / 4) + 4 half + i % 4 of the tile — are exactly those it feeds back.  F32: true fp32 products
// (v_mfma_f32_32x32x2_f32), else bf16 operands with fp32 accumulation; scores and weights are fp32 in both.  Tiles lie at multiples
// of 32 positions.
template <bool F32, int NKS, int NT>  // 16 NKS >= D, 32 NT >= V
__global__ __launch_bounds__(256, NKS <= 8 ? 2 : 1) void gate_tiles_kernel(const GateArgs a, const int* ent_start, const int* ent_len, int n_entries) {
    __shared__ float s_o[4][32][33];
    int id = blockIdx.x, e = 0, qb = 0;
    for (; e < n_entries; ++e) {
        const int nb = (ent_len[e] + 31) / 32;
        if (id < nb) {
            qb = id;
            break;
        }
        id -= nb;
    }
    if (e >= n_entries) return;
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, r = lane & 31, hf = lane >> 5;
    const int h = blockIdx.y, g = h / (a.H / a.G), D = a.D, V = a.V;
    const int m0 = ent_start[e] + 32 * qb, nq = min(32, ent_len[e] - 32 * qb);
    const int pos0 = a.row_pos[m0], qpos = pos0 + r, last = pos0 + nq - 1;
    const int my_first = first_key(qpos, a.mask);
    const int* pages = a.page_table + (size_t)a.row_slot[m0] * a.max_pages;
    const size_t cstride = (size_t)a.G * (D + V);
    const bool vec = D % 8 == 0 && V % 4 == 0 && a.ldq % 4 == 0 && ((reinterpret_cast<uintptr_t>(a.q) | reinterpret_cast<uintptr_t>(a.cache)) & 15) == 0;
    const float hb = a.bias[h];

    // eight consecutive channels from 16 ks + 8 half of a row (beyond D: some other channels of it)
    auto load8 = [&](const float* p, int ks, float (&x)[8]) {
        int d = 16 * ks + 8 * hf;
        asm volatile("" : "+v"(d));  // (worked out where it is used: kept across the tiles, all the offsets would not fit the registers)
        if (vec) {
            const float* s = p + (d < D ? d : 0);
            const f32x4 lo = *reinterpret_cast<const f32x4*>(s), hi = *reinterpret_cast<const f32x4*>(s + 4);
            x[0] = lo.x; x[1] = lo.y; x[2] = lo.z; x[3] = lo.w;
            x[4] = hi.x; x[5] = hi.y; x[6] = hi.z; x[7] = hi.w;
        } else {
#pragma unroll
            for (int u = 0; u < 8; ++u) x[u] = p[min(d + u, D - 1)];
        }
    };
    auto pack8 = [&](const float* x) {
        u32x4 pk;
        pk.x = cvt_pk_bf16(x[0], x[1]);
        pk.y = cvt_pk_bf16(x[2], x[3]);
        pk.z = cvt_pk_bf16(x[4], x[5]);
        pk.w = cvt_pk_bf16(x[6], x[7]);
        return __builtin_bit_cast(bf16x8, pk);
    };

    float qf[F32 ? NKS : 1][8];
    bf16x8 qb8[F32 ? 1 : NKS];
    {
        const float* qr = a.q + (size_t)(m0 + min(r, nq - 1)) * a.ldq + (size_t)h * D;
#pragma unroll
        for (int ks = 0; ks < NKS; ++ks) {
            float x[8];
            load8(qr, ks, x);
#pragma unroll
            for (int u = 0; u < 8; ++u) x[u] = 16 * ks + 8 * hf + u < D ? x[u] : 0.0f;  // what a key holds there then counts nothing
            if constexpr (F32) {
#pragma unroll
                for (int u = 0; u < 8; ++u) qf[ks][u] = x[u];
            } else {
                qb8[ks] = pack8(x);
            }
        }
    }
    f32x16 o[NT];
#pragma unroll
    for (int t = 0; t < NT; ++t)
#pragma unroll
        for (int i = 0; i < 16; ++i) o[t][i] = 0.0f;

    const int blk_first = first_key(pos0, a.mask), kt_lo = blk_first / 32, kt_hi = last / 32;
    for (int kt = kt_lo + wave; kt <= kt_hi; kt += 4) {
        // (positions behind the block's last row hold nothing yet, those in front of its first row's keys perhaps nothing any more)
        const int j = min(max(32 * kt + r, blk_first), last);
        const int crow = cache_row(pages, j, a.page_tokens, a.max_pages);
        const float* kp = a.cache + (size_t)crow * cstride + (size_t)g * D;
        f32x16 sc;
#pragma unroll
        for (int i = 0; i < 16; ++i) sc[i] = 0.0f;
#pragma unroll
        for (int ks = 0; ks < NKS; ++ks) {
            if (16 * ks >= D) break;
            float x[8];
            load8(kp, ks, x);
            if constexpr (F32) {
#pragma unroll
                for (int u = 0; u < 8; ++u) sc = __builtin_amdgcn_mfma_f32_32x32x2f32(x[u], qf[ks][u], sc, 0, 0, 0);
            } else {
                sc = __builtin_amdgcn_mfma_f32_32x32x16_bf16(pack8(x), qb8[ks], sc, 0, 0, 0);
            }
            if (NKS > 4 && (ks & 3) == 3) __builtin_amdgcn_sched_barrier(0);  // (large heads: what is requested together fits the registers)
        }
        float p[16];
        const float* vrow[16];
#pragma unroll
        for (int i = 0; i < 16; ++i) {
            const int kl = 8 * (i >> 2) + 4 * hf + (i & 3), key = 32 * kt + kl;
            vrow[i] = a.cache + (size_t)__shfl(crow, kl, 64) * cstride + (size_t)a.G * D + (size_t)g * V;
            const float z = fmaf(sc[i], a.scale, hb);
            const float w = F32 ? 1.0f / (1.0f + expf(-z)) : __builtin_amdgcn_rcpf(1.0f + __expf(-z));
            p[i] = key <= qpos && key >= my_first && r < nq ? w : 0.0f;
        }
        bf16x8 pf0, pf1;
        if constexpr (!F32) {
            pf0 = pack8(p);
            pf1 = pack8(p + 8);
        }
#pragma unroll
        for (int t = 0; t < NT; ++t) {
            if (32 * t >= V) break;
            const int c = min(32 * t + r, V - 1);
            float v[16];
#pragma unroll
            for (int i = 0; i < 16; ++i) v[i] = vrow[i][c];
            if constexpr (F32) {
#pragma unroll
                for (int i = 0; i < 16; ++i) o[t] = __builtin_amdgcn_mfma_f32_32x32x2f32(v[i], p[i], o[t], 0, 0, 0);
            } else {
                o[t] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(pack8(v), pf0, o[t], 0, 0, 0);
                o[t] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(pack8(v + 8), pf1, o[t], 0, 0, 0);
            }
            if (NT > 2 && (t & 1)) __builtin_amdgcn_sched_barrier(0);
        }
    }
    // the four waves' sums, 32 channels at a time: accumulator element i is channel 8 (i / 4) + 4 half + i % 4 of query r
#pragma unroll
    for (int t = 0; t < NT; ++t) {
        if (32 * t >= V) break;
        __syncthreads();
#pragma unroll
        for (int i = 0; i < 16; ++i) s_o[wave][r][8 * (i >> 2) + 4 * hf + (i & 3)] = o[t][i];
        __syncthreads();
        for (int x = tid; x < 32 * 32; x += 256) {
            const int row = x >> 5, c = x & 31;
            if (row < nq && 32 * t + c < V)
                a.out[(size_t)(m0 + row) * a.ldo + (size_t)h * V + 32 * t + c] = (s_o[0][row][c] + s_o[1][row][c]) + (s_o[2][row][c] + s_o[3][row][c]);
        }
    }
}

constexpr int kGateSpread = 512;  // (rows x heads x shares) up to which every head gets a workgroup of its own
constexpr int kGateShare = 512;  // keys of a row that one workgroup walks: up to there no partial sums are written

int gate_splits(int key_capacity) { return std::max(1, std::min(kWinSplits, (key_capacity + kGateShare - 1) / kGateShare)); }

}  // namespace

size_t gate_split_workspace(int H, int V, int key_capacity) {
    const int n = gate_splits(key_capacity);
    return n > 1 ? (size_t)kGemvMaxRows * n * H * V : 0;
}

int launch_gate_attention(const float* q, int ldq, float* out, int ldo, int M, int H, int G, int D, int V, float scale, const float* bias, KeyMask mask,
                          bool f32, const Rotary* rot, const ValuePrep& vals, const int* row_pos, const int* row_slot, const int* page_table,
                          int max_pages, int page_tokens, float* cache, int key_capacity, float* ws, size_t ws_floats, const int* ent_start,
                          const int* ent_len, int n_entries, hipStream_t s, bool* taken) {
    *taken = false;
    if (M <= 0) return ZG_OK;
    ZG_REQUIRE(H >= 1 && G >= 1 && H % G == 0 && bias && mask.keep == 0, ZG_ERR_ARG, "attention with sigmoid weights: %d heads on %d key heads", H, G);
    if (const char* e = getenv("ZGPT2_LM_WINDOW_GENERAL"))  // test hook: every step through the general kernel
        if (atoi(e) != 0) return ZG_OK;
    if (D > 256 || V > 256) return ZG_OK;  // the general kernel takes it
    GateArgs a;
    a.q = q; a.ldq = ldq; a.out = out; a.ldo = ldo; a.H = H; a.G = G; a.D = D; a.V = V; a.scale = scale; a.bias = bias; a.mask = mask;
    a.row_pos = row_pos; a.row_slot = row_slot; a.page_table = page_table; a.max_pages = max_pages; a.page_tokens = page_tokens; a.cache = cache;
    if (M > kGemvMaxRows) {
        ZG_REQUIRE(!rot && ent_start && ent_len, ZG_ERR_ARG, "attention with sigmoid weights: a portion's rows are prepared in front of it");
        const dim3 grid((M + 31) / 32 + n_entries, H);
        const int need = std::max(D, V);
#define ZG_GATE_T(NKS_, NT_)                                                                          \
    do {                                                                                              \
        if (f32) gate_tiles_kernel<true, NKS_, NT_><<<grid, 256, 0, s>>>(a, ent_start, ent_len, n_entries); \
        else gate_tiles_kernel<false, NKS_, NT_><<<grid, 256, 0, s>>>(a, ent_start, ent_len, n_entries);    \
    } while (0)
        if (need <= 64) ZG_GATE_T(4, 2);
        else if (need <= 128) ZG_GATE_T(8, 4);
        else ZG_GATE_T(16, 8);
#undef ZG_GATE_T
        ZG_HIP(hipGetLastError());
        *taken = true;
        return ZG_OK;
    }
    int n_split = gate_splits(key_capacity);
    if (n_split > 1 && (!ws || (size_t)M * n_split * H * V > ws_floats)) n_split = 1;
    const int nh = M * H * n_split <= kGateSpread ? 1 : 4;
    const dim3 grid(n_split, M, G * ((H / G + nh - 1) / nh));
    ZG_REQUIRE(grid.z <= 65535, ZG_ERR_UNSUPPORTED, "attention with sigmoid weights: %d heads", H);
    const int need = std::max(D, V);
#define ZG_GATE_P(KC_, VC_, U_, NH_)                                                                                                \
    do {                                                                                                                            \
        if (rot) gate_rows_kernel<KC_, VC_, U_, NH_, true><<<grid, 64 * kGateWaves, 0, s>>>(a, *rot, vals, ws);                     \
        else gate_rows_kernel<KC_, VC_, U_, NH_, false><<<grid, 64 * kGateWaves, 0, s>>>(a, Rotary{nullptr, 0, 1.0f}, vals, ws);    \
    } while (0)
#define ZG_GATE_R(KC_, VC_, U1_, U4_)             \
    do {                                          \
        if (nh == 1) ZG_GATE_P(KC_, VC_, U1_, 1); \
        else ZG_GATE_P(KC_, VC_, U4_, 4);         \
    } while (0)
    if (need <= 64) ZG_GATE_R(8, 1, 4, 2);
    else if (need <= 128) ZG_GATE_R(16, 2, 2, 1);
    else ZG_GATE_R(32, 4, 1, 1);
#undef ZG_GATE_P
#undef ZG_GATE_R
    ZG_HIP(hipGetLastError());
    if (n_split > 1) {
        gate_merge_kernel<<<dim3(M, (H * V + 255) / 256), 256, 0, s>>>(ws, n_split, out, ldo, H * V);
        ZG_HIP(hipGetLastError());
    }
    *taken = true;
    return ZG_OK;
}

}  // namespace lm
}  // namespace zg
