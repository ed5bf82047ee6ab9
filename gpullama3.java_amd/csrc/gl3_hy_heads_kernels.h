// gl3_hy_heads_kernels.h — kernels of two further mixers of the layer-list family: softmax attention whose heads' scores are scaled per head,
// capped and mixed with each other inside chunks of the sequence, and the gated delta rule (short convolutions, unit keys, a matrix memory
// that writes what the key does not already recall).  Every mechanism takes its sizes and constants as arguments.
#pragma once
#include "gl3_hy_kernels.h"

typedef float hy_v4f __attribute__((ext_vector_type(4)));

// ---- attention over all heads at once -----------------------------------------------------------------------------------------------
// s[h][i][j] = scale (q_ih . k_jg) (temp[h]) ; s <- cap tanh(s / cap) ; s[h] <- sum_g mix[h][g] s[g] ; key j is seen by query i if j <= i and both
// lie in the same run of `chunk` positions (chunk <= 0: every earlier key).  Because a mixed score needs every head's score of the same
// (query, key), a workgroup owns ALL heads of QT tokens for the whole walk over its key tiles (KT = 16 KB keys each):
//   1  scores: per key / value head the rows (token, head of the group) in blocks of 16 against 16 KB keys, v_mfma_f32_16x16x4_f32 on operands
//      read straight from the caches (a lane takes four consecutive entries of its row, which serve four products: the order in which a
//      product sums its k is free; the loads of CB such pieces are issued together); scaled, tempered and capped into LDS, S[head][token][key]
//   2  mixing: [H x H] (staged in LDS once) times S in place, a wavefront per (token, 16 keys), and the mask
//   3  running maximum, denominator and weights per (head, token)
//   4  weighted values: S[rows][keys] times V, accumulated in registers: a unit = 16 rows x 64 value columns of one key / value head
// Value units past what the eight wavefronts hold in registers go to further workgroups (blockIdx.y), which make the scores again.  Splits
// over the keys (blockIdx.z) write (max, denominator, unnormalised sum) per (token, head, split) for hy_attn_merge_kernel.
struct HyHeadsArgs {
    const float* q; int ldq;            // q of (t, h): q + t ldq + h dk
    const float* kc; const float* vc;   // slot-relative cache bases; row j of head g: kc + j G dk + g dk, vc + j G dv + g dv
    size_t slot_stride;
    int H, G, dk, dv;
    float scale, cap;                   // cap <= 0: none
    const float* temp;                  // [H]; null: none
    const float* mixT; int mix_ld;      // transposed mixing matrix [g][h], rows of mix_ld = H rounded up to 16, zero padded; null: none
    int chunk;
    const int* dyn; int n, nsplit;
    float* part_acc; float* part_ml;    // [n][H][nsplit][dv], [n][H][nsplit][2]
    int QT, ts, ss;                     // tokens per workgroup; LDS strides of a token's keys and of a head
    int ug;                             // value units per blockIdx.y
};
constexpr int HY_HEADS_MAX = 128;       // heads (mixing: 8 row blocks of 16)

// four consecutive entries c .. c + 3 of a row of `len`.  VEC: the rows allow 16-byte loads and c + 3 < len; else element by element, zero behind the row
template <bool VEC>
__device__ __forceinline__ hy_v4f hy_row4(const float* __restrict__ row, int c, int len) {
    if constexpr (VEC) return *reinterpret_cast<const hy_v4f*>(row + c);
    hy_v4f v = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
    for (int i = 0; i < 4; ++i)
        if (c + i < len) v[i] = row[c + i];
    return v;
}

// VEC: dk a multiple of 16, dv of 4, queries and cache rows 16-byte aligned
template <int KB, int UA, bool VEC>
static __global__ __launch_bounds__(512) void hy_heads_attn_kernel(HyHeadsArgs a) {
    extern __shared__ __attribute__((aligned(16))) float smem[];
    constexpr int KT = 16 * KB, NW = 8, NT = 64 * NW, CB = !VEC ? 1 : KB == 1 ? 8 : KB == 2 ? 4 : 2;
    const int H = a.H, G = a.G, dk = a.dk, dv = a.dv, QT = a.QT, ts = a.ts, ss = a.ss, hpg = H / G;
    float* S = smem;                       // [H][ss]: token at stride ts, KT keys
    float* sM = S + (size_t)H * ss;        // [H QT] running maximum, denominator, correction of the tile
    float* sL = sM + H * QT;
    float* sC = sL + H * QT;
    float* sT = sC + H * QT;               // [H][mix_ld] transposed mixing matrix
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), i16 = lane & 15, kq = lane >> 4;
    const int t0 = ((int)gridDim.x - 1 - (int)blockIdx.x) * QT, split = blockIdx.z;      // late tokens (most keys) first
    const int nt = min(QT, a.n - t0), pos0 = a.dyn[0], p0 = pos0 + t0, maxpos = p0 + nt - 1;
    const size_t slot = (size_t)a.dyn[1] * a.slot_stride;
    const float *kc = a.kc + slot, *vc = a.vc + slot;
    const int ldk = G * dk, ldv = G * dv, R = QT * hpg, RB = (R + 15) >> 4, CG = (dv + 63) >> 6;
    const int lo = a.chunk > 0 ? p0 / a.chunk * a.chunk : 0;       // first key any token of the workgroup sees
    const int lo_t = lo / KT, nv = maxpos / KT - lo_t + 1;
    for (int i = tid; i < H * QT; i += NT) { sM[i] = -INFINITY; sL[i] = 0.f; }
    if (a.mixT)
        for (int i = tid; i < H * a.mix_ld; i += NT) sT[i] = a.mixT[i];
    const int u0 = blockIdx.y * a.ug, u_end = min(u0 + a.ug, G * RB * CG);
    // the wavefront's value units: key / value head, row block, first column
    constexpr bool EARLY = VEC && KB == 1 && UA <= 2;          // a tile's value rows fit beside everything else: they are fetched with its keys
    int ug[UA], ur[UA], uc[UA];
    hy_v4f acc[UA][4], ve[EARLY ? UA : 1][4];
#pragma unroll
    for (int u = 0; u < UA; ++u) {
        const int unit = min(u0 + wave * UA + u, G * RB * CG - 1), rem = unit % (RB * CG);
        ug[u] = unit / (RB * CG); ur[u] = rem / CG * 16; uc[u] = rem % CG * 64;
#pragma unroll
        for (int e = 0; e < 4; ++e) acc[u][e] = hy_v4f{0.f, 0.f, 0.f, 0.f};
    }
    auto value_row = [&](int u, int j) { return vc + (size_t)min(j, maxpos) * ldv + (size_t)ug[u] * dv; };
    auto value_col = [&](int u) { return VEC ? min(uc[u] + 4 * i16, dv - 4) : uc[u] + 4 * i16; };          // (columns past dv are not stored)
    for (int vt = split; vt < nv; vt += a.nsplit) {
        const int j0 = (lo_t + vt) * KT;
        if constexpr (EARLY)
#pragma unroll
            for (int u = 0; u < UA; ++u)
#pragma unroll
                for (int i = 0; i < 4; ++i) ve[u][i] = hy_row4<VEC>(value_row(u, j0 + 4 * kq + i), value_col(u), dv);
        __syncthreads();                   // the previous tile's weights are consumed
        // 1: scores
        for (int task = wave; task < G * RB; task += NW) {
            const int g = task / RB, rb = task - g * RB;
            const int rho = rb * 16 + i16, rr = rho < R ? rho : 0, tok = min(rr / hpg, nt - 1), hh = g * hpg + rr % hpg;
            const float* qr = a.q + (size_t)(t0 + tok) * a.ldq + (size_t)hh * dk;
            const float* kr[KB];
            hy_v4f sc[KB];
#pragma unroll
            for (int b = 0; b < KB; ++b) {
                kr[b] = kc + (size_t)min(j0 + 16 * b + i16, maxpos) * ldk + (size_t)g * dk;
                sc[b] = hy_v4f{0.f, 0.f, 0.f, 0.f};
            }
            for (int c0 = 0; c0 < dk; c0 += 16 * CB) {
                hy_v4f qv[CB], kv[CB][KB];
#pragma unroll
                for (int x = 0; x < CB; ++x) {
                    if (c0 + 16 * x >= dk) break;
                    const int c = c0 + 16 * x + 4 * kq;
                    qv[x] = hy_row4<VEC>(qr, c, dk);
#pragma unroll
                    for (int b = 0; b < KB; ++b) kv[x][b] = hy_row4<VEC>(kr[b], c, dk);
                }
#pragma unroll
                for (int x = 0; x < CB; ++x) {
                    if (c0 + 16 * x >= dk) break;
#pragma unroll
                    for (int i = 0; i < 4; ++i)
#pragma unroll
                        for (int b = 0; b < KB; ++b) sc[b] = __builtin_amdgcn_mfma_f32_16x16x4f32(qv[x][i], kv[x][b][i], sc[b], 0, 0, 0);
                }
            }
#pragma unroll
            for (int r = 0; r < 4; ++r) {  // the lane holds rows 4 kq + r of column i16
                const int ro = rb * 16 + 4 * kq + r;
                if (ro >= R) continue;
                const int tk = ro / hpg, hd = g * hpg + ro % hpg, p = p0 + tk;
                const float mul = a.scale * (a.temp ? a.temp[hd] : 1.f);
                const int lo_p = a.chunk > 0 ? p / a.chunk * a.chunk : 0;
#pragma unroll
                for (int b = 0; b < KB; ++b) {
                    float s = sc[b][r] * mul;
                    if (a.cap > 0.f) s = a.cap * tanhf(s / a.cap);
                    if (!a.mixT) {
                        const int j = j0 + 16 * b + i16;
                        if (tk >= nt || j > p || j < lo_p) s = -INFINITY;
                    }
                    S[hd * ss + tk * ts + 16 * b + i16] = s;
                }
            }
        }
        __syncthreads();
        // 2: mixing and mask
        if (a.mixT) {
            const int MB = a.mix_ld >> 4;
            for (int nb = wave; nb < QT * KB; nb += NW) {
                const int tk = nb / KB, b = nb - tk * KB;
                float* col = S + tk * ts + 16 * b + i16;
                hy_v4f m[8];
#pragma unroll
                for (int mb = 0; mb < 8; ++mb) m[mb] = hy_v4f{0.f, 0.f, 0.f, 0.f};
                for (int g0 = 0; g0 < H; g0 += 4) {
                    const int g = g0 + kq;
                    const float sv = g < H ? col[g * ss] : 0.f;
                    const float* tr = sT + min(g, H - 1) * a.mix_ld + i16;
#pragma unroll
                    for (int mb = 0; mb < 8; ++mb)
                        if (mb < MB) m[mb] = __builtin_amdgcn_mfma_f32_16x16x4f32(tr[16 * mb], sv, m[mb], 0, 0, 0);
                }
                const int p = p0 + tk, j = j0 + 16 * b + i16, lo_p = a.chunk > 0 ? p / a.chunk * a.chunk : 0;
                const bool seen = tk < nt && j <= p && j >= lo_p;
#pragma unroll
                for (int mb = 0; mb < 8; ++mb)
                    if (mb < MB) {
#pragma unroll
                        for (int r = 0; r < 4; ++r) {
                            const int hd = 16 * mb + 4 * kq + r;
                            if (hd < H) col[hd * ss] = seen ? m[mb][r] : -INFINITY;
                        }
                    }
            }
            __syncthreads();
        }
        // 3: four lanes per (head, token) row, KB pieces of four keys each
        for (int row = tid >> 2; row < H * QT; row += NT / 4) {
            const int hd = row / QT, tk = row - hd * QT;
            float* sr = S + hd * ss + tk * ts + 4 * (tid & 3);
            hy_v4f v[KB];
            float mx = -INFINITY;
#pragma unroll
            for (int b = 0; b < KB; ++b) {
                v[b] = *reinterpret_cast<const hy_v4f*>(sr + 16 * b);
                mx = fmaxf(mx, fmaxf(fmaxf(v[b][0], v[b][1]), fmaxf(v[b][2], v[b][3])));
            }
            mx = fmaxf(mx, __shfl_xor(mx, 1, 64));
            mx = fmaxf(mx, __shfl_xor(mx, 2, 64));
            const float mo = sM[row], mn = fmaxf(mo, mx);
            const bool any = mn > -INFINITY;                       // false: the row has seen no key yet
            float sum = 0.f;
#pragma unroll
            for (int b = 0; b < KB; ++b) {
#pragma unroll
                for (int i = 0; i < 4; ++i) { v[b][i] = any ? expf(v[b][i] - mn) : 0.f; sum += v[b][i]; }
                *reinterpret_cast<hy_v4f*>(sr + 16 * b) = v[b];
            }
            sum += __shfl_xor(sum, 1, 64);
            sum += __shfl_xor(sum, 2, 64);
            if ((tid & 3) == 0) {
                const float corr = any ? expf(mo - mn) : 1.f;      // exp(-inf) = 0 the first time
                sM[row] = mn; sL[row] = sL[row] * corr + sum; sC[row] = corr;
            }
        }
        __syncthreads();
        // 4: weighted values
#pragma unroll
        for (int u = 0; u < UA; ++u) {
            if (u0 + wave * UA + u >= u_end) continue;
            const int g = ug[u];
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                const int ro = ur[u] + 4 * kq + r;
                const float c = ro < R ? sC[(g * hpg + ro % hpg) * QT + ro / hpg] : 0.f;
#pragma unroll
                for (int e = 0; e < 4; ++e) acc[u][e][r] *= c;
            }
            const int rho = ur[u] + i16;
            const float* pr = S + (size_t)(g * hpg + (rho < R ? rho % hpg : 0)) * ss + (rho < R ? rho / hpg : 0) * ts + 4 * kq;
            hy_v4f v4[KB][4];
#pragma unroll
            for (int b = 0; b < KB; ++b)
#pragma unroll
                for (int i = 0; i < 4; ++i) {
                    if constexpr (EARLY) v4[b][i] = ve[u][i];
                    else v4[b][i] = hy_row4<VEC>(value_row(u, j0 + 16 * b + 4 * kq + i), value_col(u), dv);
                }
#pragma unroll
            for (int b = 0; b < KB; ++b) {
                hy_v4f pv = *reinterpret_cast<const hy_v4f*>(pr + 16 * b);
                if (rho >= R) pv = hy_v4f{0.f, 0.f, 0.f, 0.f};
#pragma unroll
                for (int i = 0; i < 4; ++i)
#pragma unroll
                    for (int e = 0; e < 4; ++e) acc[u][e] = __builtin_amdgcn_mfma_f32_16x16x4f32(pv[i], v4[b][i][e], acc[u][e], 0, 0, 0);
            }
        }
    }
    __syncthreads();
    if (blockIdx.y == 0)
        for (int row = tid; row < H * nt; row += NT) {
            const int tk = row / H, hd = row - tk * H;
            const size_t o = ((size_t)(t0 + tk) * H + hd) * a.nsplit + split;
            a.part_ml[2 * o] = sM[hd * QT + tk]; a.part_ml[2 * o + 1] = sL[hd * QT + tk];
        }
#pragma unroll
    for (int u = 0; u < UA; ++u) {
        if (u0 + wave * UA + u >= u_end) continue;
        const int c = uc[u] + 4 * i16;
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const int ro = ur[u] + 4 * kq + r, tk = ro / hpg;
            if (ro >= R || tk >= nt) continue;
            float* dst = a.part_acc + (((size_t)(t0 + tk) * H + ug[u] * hpg + ro % hpg) * a.nsplit + split) * dv;
            if constexpr (VEC) {
                if (c < dv) *reinterpret_cast<hy_v4f*>(dst + c) = hy_v4f{acc[u][0][r], acc[u][1][r], acc[u][2][r], acc[u][3][r]};
            } else {
#pragma unroll
                for (int e = 0; e < 4; ++e)
                    if (c + e < dv) dst[c + e] = acc[u][e][r];
            }
        }
    }
}

// ---- gated delta rule ---------------------------------------------------------------------------------------------------------------
// What enters the recurrence, one wavefront per (token, head of q | k | v): the causal depthwise convolution over time (hy_conv_row), silu
// (act), for q and k x / sqrt(sum x^2 + 1e-6) (unit) times a multiplier, written to out [n][C] in the order of the projection row.  The last
// blockIdx.y makes the gates: ga = exp(-exp(A_log) softplus(z_a + dt_bias)), gb = sigmoid(z_b).
struct HyDeltaPrep {
    const float* proj; int ld, c0;      // the row's q | k | v columns start at c0
    int G, H, D, V;
    const float* conv_w; int taps;      // [taps][C], last row = current token
    float* tail; size_t slot_stride; const int* dyn; int n;
    int act, unit; float q_mul, k_mul;
    float* out;
    int a_off, b_off; const float* A_log; const float* dt_bias; float* ga; float* gb;      // [n][H]
};
static __global__ __launch_bounds__(64) void hy_delta_prep_kernel(HyDeltaPrep x) {
    __shared__ float crow[HY_PREP_MAXD];
    const int t = blockIdx.x, hh = blockIdx.y, lane = threadIdx.x;
    if (hh == 2 * x.G + x.H) {
        const float* row = x.proj + (size_t)t * x.ld;
        for (int h = lane; h < x.H; h += 64) {
            x.ga[(size_t)t * x.H + h] = expf(-expf(x.A_log[h]) * hy_softplus(row[x.a_off + h] + x.dt_bias[h]));
            x.gb[(size_t)t * x.H + h] = hy_sigmoid(row[x.b_off + h]);
        }
        return;
    }
    const bool isv = hh >= 2 * x.G;
    const int len = isv ? x.V : x.D, cc = isv ? 2 * x.G * x.D + (hh - 2 * x.G) * x.V : hh * x.D, C = 2 * x.G * x.D + x.H * x.V;
    hy_conv_row(crow, x.proj, x.ld, x.c0 + cc, t, len, x.conv_w + cc, C, x.taps, x.tail + (size_t)x.dyn[1] * x.slot_stride + cc, x.dyn[0] == 0, x.n == 1);
    float r = 1.f, ss = 0.f;
    for (int d = lane; d < len; d += 64) {          // (a lane reads back its own entries)
        const float v = x.act ? hy_silu(crow[d]) : crow[d];
        crow[d] = v;
        ss += v * v;
    }
    if (!isv) {
        if (x.unit) r = 1.f / sqrtf(hy_wave_sum(ss) + 1e-6f);
        r *= hh < x.G ? x.q_mul : x.k_mul;
    }
    float* dst = x.out + (size_t)t * C + cc;
    for (int d = lane; d < len; d += 64) dst[d] = crow[d] * r;
}

// sum over the NG neighbouring lanes that share a column (NG a power of two); every lane gets it.  Inside 16 lanes the partners are reached by
// DPP (quad permutations, then the mirrored half row and row: the parts that meet there are already equal on all lanes of a quad / half)
template <int CTRL>
__device__ __forceinline__ float hy_dpp(float v) { return __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), CTRL, 0xf, 0xf, true)); }
template <int NG>
__device__ __forceinline__ float hy_group_sum(float v) {
    if constexpr (NG >= 2) v += hy_dpp<0xB1>(v);          // quad_perm [1, 0, 3, 2]
    if constexpr (NG >= 4) v += hy_dpp<0x4E>(v);          // quad_perm [2, 3, 0, 1]
    if constexpr (NG >= 8) v += hy_dpp<0x141>(v);         // row_half_mirror
    if constexpr (NG >= 16) v += hy_dpp<0x140>(v);        // row_mirror
    if constexpr (NG >= 32) v += __shfl_xor(v, 16, 64);
    if constexpr (NG >= 64) v += __shfl_xor(v, 32, 64);
    return v;
}

// S <- a S; u = b (v - S^T k); S <- S + k u^T; o = S^T q, token by token.  Workgroup = one head x 4 wavefronts, a wavefront = 64 / NG value columns, a
// column's N states over NG lanes x NL registers (lane i holds the states 4 (NG j + i) .. + 3; NG NL >= N).  Tokens run in order, TB at a
// time: a block's key and query rows, values and gates come from memory into registers while the block before it is walked, then into one
// of two LDS buffers (one barrier per block); a token's slices are fetched from LDS one token ahead.  Both sums over a column's lanes stay in
// registers (hy_group_sum); lane i of a column keeps o of the tokens i, i + NG, ... and stores them at the block's end.  Tokens past
// the step's end are walked with a = 1, b = 0, which changes nothing.
struct HyDeltaScan {
    const float* src; int ld, k_off, v_off;            // rows q | k | v as hy_delta_prep_kernel leaves them (q at 0)
    const float* ga; const float* gb;                  // [n][heads]
    int heads, G, P, N;
    float* state; size_t slot_stride; const int* dyn; int n;      // [heads][N][P] per slot
    float* y; int ldy;
};
template <int NL, int NG>
static __global__ __launch_bounds__(256) void hy_delta_scan_kernel(HyDeltaScan a) {
    constexpr int Ns = NL * NG, cpw = 64 / NG, cols = 4 * cpw, NQ = NL / 4, TB = Ns <= 128 ? 16 : Ns <= 256 ? 8 : Ns <= 512 ? 4 : 2;
    constexpr int pieces = TB * Ns / 2, NP = (pieces + 255) / 256, NV = (TB * cols + 255) / 256, YR = TB > NG ? TB / NG : 1;
    __shared__ __attribute__((aligned(16))) float sKQ[2][TB * 2 * Ns];      // [token][key Ns | query Ns]
    __shared__ float sV[2][TB * cols];
    __shared__ float2 sG[2][TB];
    const int P = a.P, N = a.N, n = a.n;
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, head = blockIdx.y, ng = lane % NG;
    const int col0 = blockIdx.x * cols, myc = wave * cpw + lane / NG, p = col0 + myc;
    const bool livep = p < P;
    const int g = head / (a.heads / a.G);
    const float *qbase = a.src + (size_t)g * N, *kbase = qbase + a.k_off, *vbase = a.src + a.v_off + (size_t)head * P;
    const bool vec = (N & 3) == 0 && (a.ld & 3) == 0 && (((uintptr_t)qbase | (uintptr_t)kbase) & 15) == 0;
    float* S = a.state + (size_t)a.dyn[1] * a.slot_stride + (size_t)head * N * P;
    const bool fresh = a.dyn[0] == 0;
    hy_v4f s[NQ];
#pragma unroll
    for (int j = 0; j < NQ; ++j)
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            const int nn = 4 * (NG * j + ng) + e;
            s[j][e] = (!fresh && livep && nn < N) ? S[(size_t)nn * P + p] : 0.f;
        }
    hy_v4f rk[NP];
    float rv[NV];
    float2 rg;
    auto load = [&](int t0) {
#pragma unroll
        for (int u = 0; u < NP; ++u) {
            const int i = tid + u * 256, t = min(t0 + i / (Ns / 2), n - 1), c = i % (Ns / 2) * 4;
            const bool isq = c >= Ns;
            const float* row = (isq ? qbase : kbase) + (size_t)t * a.ld;
            const int nn = isq ? c - Ns : c;
            if (vec) {
                rk[u] = *reinterpret_cast<const hy_v4f*>(row + min(nn, N - 4));
                if (nn >= N) rk[u] = hy_v4f{0.f, 0.f, 0.f, 0.f};
            } else {
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    rk[u][e] = row[min(nn + e, N - 1)];
                    if (nn + e >= N) rk[u][e] = 0.f;
                }
            }
        }
#pragma unroll
        for (int u = 0; u < NV; ++u) {
            const int i = tid + u * 256;
            rv[u] = vbase[(size_t)min(t0 + i / cols, n - 1) * a.ld + min(col0 + i % cols, P - 1)];
        }
        const size_t gt = (size_t)min(t0 + tid % TB, n - 1) * a.heads + head;
        rg = t0 + tid % TB < n ? make_float2(a.ga[gt], a.gb[gt]) : make_float2(1.f, 0.f);
    };
    load(0);
    for (int t0 = 0, buf = 0; t0 < n; t0 += TB, buf ^= 1) {
        const int tb = min(TB, n - t0);
#pragma unroll
        for (int u = 0; u < NP; ++u)
            if (tid + u * 256 < pieces) *reinterpret_cast<hy_v4f*>(sKQ[buf] + 4 * (tid + u * 256)) = rk[u];
#pragma unroll
        for (int u = 0; u < NV; ++u)
            if (tid + u * 256 < TB * cols) sV[buf][tid + u * 256] = rv[u];
        if (tid < TB) sG[buf][tid] = rg;
        __syncthreads();
        if (t0 + TB < n) load(t0 + TB);
        float yk[YR];
#pragma unroll
        for (int j = 0; j < YR; ++j) yk[j] = 0.f;
        hy_v4f k0[NQ], q0[NQ], k1[NQ], q1[NQ];
        float v0, v1;
        float2 g0, g1;
        auto fetch = [&](int t, hy_v4f* k4, hy_v4f* q4, float& v, float2& gg) {
            const hy_v4f* row = reinterpret_cast<const hy_v4f*>(sKQ[buf] + t * 2 * Ns) + ng;
#pragma unroll
            for (int j = 0; j < NQ; ++j) { k4[j] = row[NG * j]; q4[j] = row[Ns / 4 + NG * j]; }
            v = sV[buf][t * cols + myc]; gg = sG[buf][t];
        };
        auto walk = [&](int t, const hy_v4f* k4, const hy_v4f* q4, float v, float2 gg) {
            float r0 = 0.f, r1 = 0.f, a0 = 0.f, a1 = 0.f;
#pragma unroll
            for (int j = 0; j < NQ; ++j) {
                r0 = fmaf(s[j][0], k4[j][0], r0); r1 = fmaf(s[j][1], k4[j][1], r1);
                r0 = fmaf(s[j][2], k4[j][2], r0); r1 = fmaf(s[j][3], k4[j][3], r1);
            }
            const float u = gg.y * (v - gg.x * hy_group_sum<NG>(r0 + r1));
#pragma unroll
            for (int j = 0; j < NQ; ++j)
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    s[j][e] = fmaf(k4[j][e], u, gg.x * s[j][e]);
                    if (e & 1) a1 = fmaf(s[j][e], q4[j][e], a1); else a0 = fmaf(s[j][e], q4[j][e], a0);
                }
            const float o = hy_group_sum<NG>(a0 + a1);
#pragma unroll
            for (int j = 0; j < YR; ++j)
                if (t == j * NG + ng) yk[j] = o;
        };
        fetch(0, k0, q0, v0, g0);
        for (int t = 0; t < tb; t += 2) {          // (TB is even: the second token of the last pair may lie past the step's end)
            fetch(t + 1, k1, q1, v1, g1);
            walk(t, k0, q0, v0, g0);
            fetch(min(t + 2, TB - 1), k0, q0, v0, g0);
            walk(t + 1, k1, q1, v1, g1);
        }
#pragma unroll
        for (int j = 0; j < YR; ++j) {
            const int t = j * NG + ng;
            if (t < tb && livep) a.y[(size_t)(t0 + t) * a.ldy + head * P + p] = yk[j];
        }
    }
#pragma unroll
    for (int j = 0; j < NQ; ++j)
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            const int nn = 4 * (NG * j + ng) + e;
            if (livep && nn < N) S[(size_t)nn * P + p] = s[j][e];
        }
}
