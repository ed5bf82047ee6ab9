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
//      product sums its k is free); scaled, tempered and capped into LDS, S[head][token][key]
//   2  mixing: [H x H] times S in place, a wavefront per (token, 16 keys), and the mask
//   3  running maximum, denominator and weights per (head, token)
//   4  weighted values: S[rows][keys] times V, accumulated in registers: a unit = 16 rows x 64 value columns of one key / value head
// Value units past what four wavefronts hold in registers go to further workgroups (blockIdx.y), which make the scores again.  Splits
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

// four consecutive entries c .. c + 3 of a row of `len` (zero behind it); vec: rows allow 16-byte loads
__device__ __forceinline__ hy_v4f hy_row4(const float* __restrict__ row, int c, int len, bool vec) {
    hy_v4f v = {0.f, 0.f, 0.f, 0.f};
    if (vec) {
        if (c < len) v = *reinterpret_cast<const hy_v4f*>(row + c);
    } else {
#pragma unroll
        for (int i = 0; i < 4; ++i)
            if (c + i < len) v[i] = row[c + i];
    }
    return v;
}

template <int KB, int UA>
static __global__ __launch_bounds__(256) void hy_heads_attn_kernel(HyHeadsArgs a) {
    extern __shared__ __attribute__((aligned(16))) float smem[];
    constexpr int KT = 16 * KB;
    const int H = a.H, G = a.G, dk = a.dk, dv = a.dv, QT = a.QT, ts = a.ts, ss = a.ss, hpg = H / G;
    float* S = smem;                       // [H][ss]: token at stride ts, KT keys
    float* sM = S + (size_t)H * ss;        // [H QT] running maximum, denominator, correction of the tile
    float* sL = sM + H * QT;
    float* sC = sL + H * QT;
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, i16 = lane & 15, kq = lane >> 4;
    const int t0 = ((int)gridDim.x - 1 - (int)blockIdx.x) * QT, split = blockIdx.z;      // late tokens (most keys) first
    const int nt = min(QT, a.n - t0), pos0 = a.dyn[0], p0 = pos0 + t0, maxpos = p0 + nt - 1;
    const size_t slot = (size_t)a.dyn[1] * a.slot_stride;
    const float *kc = a.kc + slot, *vc = a.vc + slot;
    const int ldk = G * dk, ldv = G * dv, R = QT * hpg, RB = (R + 15) >> 4, CG = (dv + 63) >> 6;
    const bool vq = (dk & 3) == 0 && (a.ldq & 3) == 0 && ((uintptr_t)a.q & 15) == 0;
    const bool vk = (dk & 3) == 0 && ((uintptr_t)kc & 15) == 0, vv = (dv & 3) == 0 && ((uintptr_t)vc & 15) == 0;
    const int lo = a.chunk > 0 ? p0 / a.chunk * a.chunk : 0;       // first key any token of the workgroup sees
    const int lo_t = lo / KT, nv = maxpos / KT - lo_t + 1;
    for (int i = tid; i < H * QT; i += 256) { sM[i] = -INFINITY; sL[i] = 0.f; }
    const int u0 = blockIdx.y * a.ug, u_end = min(u0 + a.ug, G * RB * CG);
    hy_v4f acc[UA][4];
#pragma unroll
    for (int u = 0; u < UA; ++u)
#pragma unroll
        for (int e = 0; e < 4; ++e) acc[u][e] = hy_v4f{0.f, 0.f, 0.f, 0.f};
    for (int vt = split; vt < nv; vt += a.nsplit) {
        const int j0 = (lo_t + vt) * KT;
        __syncthreads();                   // the previous tile's weights are consumed
        // 1: scores
        for (int task = wave; task < G * RB; task += 4) {
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
            for (int c0 = 0; c0 < dk; c0 += 16) {
                const int c = c0 + 4 * kq;
                const hy_v4f qv = hy_row4(qr, c, dk, vq);
                hy_v4f kv[KB];
#pragma unroll
                for (int b = 0; b < KB; ++b) kv[b] = hy_row4(kr[b], c, dk, vk);
#pragma unroll
                for (int i = 0; i < 4; ++i)
#pragma unroll
                    for (int b = 0; b < KB; ++b) sc[b] = __builtin_amdgcn_mfma_f32_16x16x4f32(qv[i], kv[b][i], sc[b], 0, 0, 0);
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
            for (int nb = wave; nb < QT * KB; nb += 4) {
                const int tk = nb / KB, b = nb - tk * KB;
                float* col = S + tk * ts + 16 * b + i16;
                hy_v4f m[8];
#pragma unroll
                for (int mb = 0; mb < 8; ++mb) m[mb] = hy_v4f{0.f, 0.f, 0.f, 0.f};
                for (int g0 = 0; g0 < H; g0 += 4) {
                    const int g = g0 + kq;
                    const float sv = g < H ? col[g * ss] : 0.f;
                    const float* tr = a.mixT + (size_t)min(g, H - 1) * a.mix_ld + i16;
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
        for (int row = tid >> 2; row < H * QT; row += 64) {
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
            const int unit = u0 + wave * UA + u;
            if (unit >= u_end) continue;
            const int g = unit / (RB * CG), rem = unit - g * RB * CG, rb = rem / CG, cg = rem - rb * CG;
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                const int ro = rb * 16 + 4 * kq + r;
                const float c = ro < R ? sC[(g * hpg + ro % hpg) * QT + ro / hpg] : 0.f;
#pragma unroll
                for (int e = 0; e < 4; ++e) acc[u][e][r] *= c;
            }
            const int rho = rb * 16 + i16;
            const float* pr = S + (size_t)(g * hpg + (rho < R ? rho % hpg : 0)) * ss + (rho < R ? rho / hpg : 0) * ts + 4 * kq;
            const int c = cg * 64 + 4 * i16;
#pragma unroll
            for (int b = 0; b < KB; ++b) {
                hy_v4f pv = *reinterpret_cast<const hy_v4f*>(pr + 16 * b);
                if (rho >= R) pv = hy_v4f{0.f, 0.f, 0.f, 0.f};
                hy_v4f v4[4];
#pragma unroll
                for (int i = 0; i < 4; ++i) v4[i] = hy_row4(vc + (size_t)min(j0 + 16 * b + 4 * kq + i, maxpos) * ldv + (size_t)g * dv, c, dv, vv);
#pragma unroll
                for (int i = 0; i < 4; ++i)
#pragma unroll
                    for (int e = 0; e < 4; ++e) acc[u][e] = __builtin_amdgcn_mfma_f32_16x16x4f32(pv[i], v4[i][e], acc[u][e], 0, 0, 0);
            }
        }
    }
    __syncthreads();
    if (blockIdx.y == 0)
        for (int row = tid; row < H * nt; row += 256) {
            const int tk = row / H, hd = row - tk * H;
            const size_t o = ((size_t)(t0 + tk) * H + hd) * a.nsplit + split;
            a.part_ml[2 * o] = sM[hd * QT + tk]; a.part_ml[2 * o + 1] = sL[hd * QT + tk];
        }
#pragma unroll
    for (int u = 0; u < UA; ++u) {
        const int unit = u0 + wave * UA + u;
        if (unit >= u_end) continue;
        const int g = unit / (RB * CG), rem = unit - g * RB * CG, rb = rem / CG, cg = rem - rb * CG;
        const int c = cg * 64 + 4 * i16;
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const int ro = rb * 16 + 4 * kq + r, tk = ro / hpg;
            if (ro >= R || tk >= nt) continue;
            float* dst = a.part_acc + (((size_t)(t0 + tk) * H + g * hpg + ro % hpg) * a.nsplit + split) * dv;
            if ((dv & 3) == 0) {
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

// S <- a S; u = b (v - S^T k); S <- S + k u^T; o = S^T q, token by token.  Layout as hy_ssm_scan_kernel: workgroup = one head x 4 wavefronts, a
// wavefront = 64 / NG value columns, a column's N states over NG lanes x NL registers; tokens staged TB at a time, what a token reads from
// LDS is fetched one token ahead; partial sums of o per lane go to LDS and are joined once per block.
struct HyDeltaScan {
    const float* src; int ld, k_off, v_off;            // rows q | k | v as hy_delta_prep_kernel leaves them (q at 0)
    const float* ga; const float* gb;                  // [n][heads]
    int heads, G, P, N, TB;
    float* state; size_t slot_stride; const int* dyn; int n;      // [heads][N][P] per slot
    float* y; int ldy;
};
template <int NL, int NG>
static __global__ __launch_bounds__(256) void hy_delta_scan_kernel(HyDeltaScan a) {
    extern __shared__ __attribute__((aligned(16))) float smem[];
    constexpr int Ns = NL * NG, cpw = 64 / NG, cols = 4 * cpw, NQ = NL / 4;
    const int P = a.P, N = a.N, TB = a.TB, n = a.n;
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, head = blockIdx.y, ng = lane % NG;
    const int col0 = blockIdx.x * cols, myc = wave * cpw + lane / NG, p = col0 + myc;
    const bool livep = p < P;
    const int g = head / (a.heads / a.G);
    const float *qbase = a.src + (size_t)g * N, *kbase = qbase + a.k_off, *vbase = a.src + a.v_off + (size_t)head * P;
    float* sK = smem;                    // [TB + 1][Ns] (one row of slack: the fetch ahead of the last token)
    float* sQ = sK + (TB + 1) * Ns;      // [TB + 1][Ns]
    float* sY = sQ + (TB + 1) * Ns;      // [TB][256]
    float* sV = sY + TB * 256;           // [TB + 1][cols]
    float* sG = sV + (TB + 1) * cols;    // [TB + 1] a, [TB + 1] b
    float* S = a.state + (size_t)a.dyn[1] * a.slot_stride + (size_t)head * N * P;
    const bool fresh = a.dyn[0] == 0;
    float s[NL];
#pragma unroll
    for (int i = 0; i < NL; ++i) {
        const int nn = ng * NL + i;
        s[i] = (!fresh && livep && nn < N) ? S[(size_t)nn * P + p] : 0.f;
    }
    for (int t0 = 0; t0 < n; t0 += TB) {
        const int tb = min(TB, n - t0);
        __syncthreads();
        hy_scan_stage(sK, kbase, a.ld, t0, tb, N, Ns, 1.f, 0);
        hy_scan_stage(sQ, qbase, a.ld, t0, tb, N, Ns, 1.f, 0);
        for (int i = tid; i < tb * cols; i += 256) {
            const int t = i / cols, c = i - t * cols;
            sV[i] = col0 + c < P ? vbase[(size_t)(t0 + t) * a.ld + col0 + c] : 0.f;
        }
        if (tid < tb) {
            sG[tid] = a.ga[(size_t)(t0 + tid) * a.heads + head];
            sG[TB + 1 + tid] = a.gb[(size_t)(t0 + tid) * a.heads + head];
        }
        __syncthreads();
        hy_v4f kc[NQ], qc[NQ], kn[NQ], qn[NQ];
        float vc, gc, bc, vn, gn, bn;
        auto fetch = [&](int t, hy_v4f* k4, hy_v4f* q4, float& v, float& ga, float& gb) {
            const hy_v4f* ks = reinterpret_cast<const hy_v4f*>(sK + t * Ns + ng * NL);
            const hy_v4f* qs = reinterpret_cast<const hy_v4f*>(sQ + t * Ns + ng * NL);
#pragma unroll
            for (int i = 0; i < NQ; ++i) { k4[i] = ks[i]; q4[i] = qs[i]; }
            v = sV[t * cols + myc]; ga = sG[t]; gb = sG[TB + 1 + t];
        };
        fetch(0, kc, qc, vc, gc, bc);
        for (int t = 0; t < tb; ++t) {
            fetch(t + 1, kn, qn, vn, gn, bn);
            float r0 = 0.f, r1 = 0.f;
#pragma unroll
            for (int i = 0; i < NQ; ++i) {
                r0 = fmaf(s[4 * i], kc[i][0], r0); r1 = fmaf(s[4 * i + 1], kc[i][1], r1);
                r0 = fmaf(s[4 * i + 2], kc[i][2], r0); r1 = fmaf(s[4 * i + 3], kc[i][3], r1);
            }
            const float rec = hy_group_sum<NG>(r0 + r1);
            const float u = bc * (vc - gc * rec);
            float a0 = 0.f, a1 = 0.f;
#pragma unroll
            for (int i = 0; i < NQ; ++i)
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    float& st = s[4 * i + e];
                    st = fmaf(kc[i][e], u, gc * st);
                    if (e & 1) a1 = fmaf(st, qc[i][e], a1); else a0 = fmaf(st, qc[i][e], a0);
                }
            sY[t * 256 + tid] = a0 + a1;
#pragma unroll
            for (int i = 0; i < NQ; ++i) { kc[i] = kn[i]; qc[i] = qn[i]; }
            vc = vn; gc = gn; bc = bn;
        }
        __syncthreads();
        for (int i = tid; i < tb * cols; i += 256) {
            const int t = i / cols, c = i - t * cols;
            if (col0 + c >= P) continue;
            float v = 0.f;
#pragma unroll 4
            for (int k = 0; k < NG; ++k) v += sY[t * 256 + c * NG + k];
            a.y[(size_t)(t0 + t) * a.ldy + head * P + col0 + c] = v;
        }
    }
#pragma unroll
    for (int i = 0; i < NL; ++i) {
        const int nn = ng * NL + i;
        if (livep && nn < N) S[(size_t)nn * P + p] = s[i];
    }
}
