// The recurrences of recurrence.hip over long portions, chunk by chunk, on the matrix units in 32-bit
// (v_mfma_f32_16x16x4_f32: IEEE 32-bit products and sums, so one kernel serves both element types).
//
// A portion of a request's rows is cut into chunks; three launches: every chunk's own contribution to the state and its
// whole decay (parallel over chunks and heads); the state before every chunk, chunk after chunk, elementwise; every
// chunk's outputs from the state before it (parallel again).  A portion of one chunk needs the last alone.
//
// Inside a chunk a block (one head, up to 128 value columns) takes 16 rows at a time.  With f_t the decays of row t per
// key channel, F_t their product from the first of the 16 rows to row t, B_s their product from row s + 1 to the last, G
// over all 16, S the state before them:
//   o_t = (q_t F_t)^T S + sum_(s <= t) A[t][s] v_s            S <- diag(G) S + sum_s (k_s B_s) v_s^T
//   A[t][s] = sum_d q_t[d] k_s[d] f_(s+1)[d] ... f_t[d]
// The rows' pairs are split by halves: for t in the second half and s in the first half of an aligned block of 2h rows
// (h = 1, 2, 4, 8), the product of the decays falls apart at the block's middle into one factor of t and one of s, so A
// over those pairs is a product of two matrices; the four levels' results are masked to their pairs and added, with the
// diagonal apart.  Every factor is a product of decays (at most 1): no logarithms, no differences of sums, nothing that
// overflows however strong the decays, and no state is lost to rounding of a running sum.
//   mode 0 (one decay per head), mode 2 (a forget gate per channel): as above
//   mode 1 (a decay per channel, a bonus for the token itself): row t sees the state before it: F_t and A's products stop
//   before row t, and A[t][t] = sum_d q_t[d] u[d] k_t[d]
//   mode 3 (decays formed beforehand): as mode 2
//   modes 4 and 5 (one decay a row and head): A is the product of the rows' q and k, each entry times its product of
//   decays, which a lane forms for its four entries by one walk over the 16 rows; mode 5 carries n beside S (the preparing
//   waves hold it for their channels) and divides row t's outputs by max(|q_t F_t . n + sum_s A[t][s]|, fl_t) + 1e-6
//
// Preparing 16 rows is vector arithmetic, using them is matrix arithmetic: between two barriers every wave prepares the
// next 16 rows and uses the last, half of the waves in the one order and half in the other, so that the two waves that
// share a SIMD keep both of its units busy.
// Wave w prepares 16 key channels (a lane holds row r = lane % 16 of channels 4 g + j, g = lane / 16: the operand layout of
// the matrix instruction, in which a level's matrix is both operands; products along the rows run over the 16 lanes by
// register moves), leaves q F, k B, G and its share of A in shared memory (two buffers in turn, one barrier per 16 rows),
// and takes 16 value columns of the rows prepared before: the state of those columns stays in its registers, as accumulators of the state's update
// and, as they lie, as the operand of the output's product.
// With a norm behind it (a head's columns in one block), the waves leave the squares' sums of 16 rows in shared memory
// before the barrier and write the rows, normed, after it.
// chunks: int32 [n][3] = (first row, rows, 1 if the portion is this chunk alone); portions: int32 [m][3] = (first chunk,
// chunks, first row); a portion's state row is tok_seq of its first row, read on the device (a recorded step serves
// another request at every replay).  The order of all sums depends on a row's place in its portion alone.
#pragma once
#include "recurrence_gates.h"
#include <type_traits>

typedef __attribute__((ext_vector_type(4))) float floatx4;

// The workspace: [chunks][H][D][Dv] states, [chunks][H][D] decays, and in mode 5 [chunks][H][D] n.
__device__ __forceinline__ float* rec_ws_g(const Rec& a) { return a.ws + (long)a.n_chunks * a.H * a.D * a.Dv; }
__device__ __forceinline__ float* rec_ws_n(const Rec& a) { return rec_ws_g(a) + (long)a.n_chunks * a.H * a.D; }

// the value of the lane's partner in the other half of an aligned group of 2 H lanes of its 16 (for H = 4, 8 of some lane
// of that half: the callers' values are the same throughout a half)
template <int H>
__device__ __forceinline__ float other_half(float v) {
    constexpr int ctrl = H == 1 ? 0xB1 : (H == 2 ? 0x4E : (H == 4 ? 0x141 : 0x140));   // quad_perm 1032, 2301, half mirror, mirror
    return __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, v), ctrl, 0xf, 0xf, true));
}

// four neighbouring elements from an address of any alignment (an element's own)
__device__ __forceinline__ void load4(const float* __restrict__ p, float (&v)[4]) {
    typedef float float4_any __attribute__((ext_vector_type(4), aligned(4)));
    const float4_any t = *(const float4_any*)p;
#pragma unroll
    for (int j = 0; j < 4; ++j) v[j] = t[j];
}
__device__ __forceinline__ void load4(const bf16_t* __restrict__ p, float (&v)[4]) {
    typedef unsigned short ushort4_any __attribute__((ext_vector_type(4), aligned(2)));
    const ushort4_any t = *(const ushort4_any*)p;
#pragma unroll
    for (int j = 0; j < 4; ++j) v[j] = bf16_bits_to_float(t[j]);
}

// What a lane brings of one tile of 16 channels for 16 rows: channels d .. d + 3 of its row.
struct RecRaw { float q[4], k[4], w[4]; };

template <typename TA, int MODE, int PHASE, int DT, int W>
__global__ __launch_bounds__(W * 64, 2) void recurrence_chunks_kernel(Rec a) {
    constexpr int DP = DT * 16, LD = DP + 4, NPT = (DT + W - 1) / W;
    __shared__ __align__(16) float qt[PHASE == 1 ? 2 : 1][16][LD];
    __shared__ __align__(16) float kt[2][16][LD];
    __shared__ __align__(16) float gt[2][DP];
    __shared__ __align__(16) float at[PHASE == 1 ? 2 : 1][W][16][20];
    __shared__ __align__(16) float sq[PHASE == 1 ? 2 : 1][W][16];
    constexpr bool SCALAR = MODE >= 4, DIV = MODE == 5;
    __shared__ __align__(16) float dnt[DIV && PHASE == 1 ? 2 : 1][W][2][16];
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, waves = blockDim.x >> 6, g = lane >> 4, r = lane & 15;
    const int c = blockIdx.x, h = blockIdx.y, hk = h / (a.H / a.Hk);
    const int row0 = a.chunks[3 * c], n = a.chunks[3 * c + 1], single = a.chunks[3 * c + 2];
    if (PHASE == 0 && single) return;
    const int H = a.H, D = a.D, Dv = a.Dv;
    const int col0 = blockIdx.z * 128 + wave * 16, col = col0 + r;
    const bool has_cols = col0 < Dv;
    const bool col_ok = has_cols && col < Dv;
    constexpr int PREP = DT < W ? DT : W;                  // waves that prepare channels (the launch has at least as many)
    const TA* q = (const TA*)a.q;
    const TA* k = (const TA*)a.k;
    const TA* v = (const TA*)a.v;
    floatx4 S[DT];
    float* slot = a.state + (long)a.tok_seq[row0] * a.state_stride + (long)h * D * Dv;
    float* mine = a.ws + ((long)c * H + h) * D * Dv;
    const float* from = single ? slot : mine;
#pragma unroll
    for (int ct = 0; ct < DT; ++ct) {
        S[ct] = floatx4{0.f, 0.f, 0.f, 0.f};
        if (PHASE == 1) {
#pragma unroll
            for (int i = 0; i < 4; ++i) {                  // (from an address that is always valid: no branch between the loads)
                const int d = ct * 16 + 4 * g + i;
                const float x = from[(d < D ? d : D - 1) * Dv + (col_ok ? col : 0)];
                S[ct][i] = col_ok && d < D ? x : 0.f;
            }
        }
    }
    // the constants of the wave's channels
    float bias[NPT][4], low[NPT][4], whole[NPT][4], nn[DIV ? NPT : 1][4];
    float* const n_slot = a.state + (long)a.tok_seq[row0] * a.state_stride + (long)H * D * Dv + (long)h * D;   // (copy z at + z * H * D)
    float* const n_mine = DIV ? rec_ws_n(a) + ((long)c * H + h) * D : nullptr;
    const float dec = MODE == 0 ? a.decay[h] : 0.f;
#pragma unroll
    for (int p = 0; p < NPT; ++p) {
        const int d0 = (wave + p * waves) * 16 + 4 * g;
#pragma unroll
        for (int j = 0; j < 4; ++j) {
            const int d = min(d0 + j, D - 1);              // (what stands beyond the head's channels is not used)
            bias[p][j] = MODE == 1 || MODE == 2 ? a.w0[h * D + d] : 0.f;
            low[p][j] = MODE == 1 || MODE == 2 ? a.u[h * D + d] : 0.f;
            whole[p][j] = 1.f;
            if (DIV) nn[p][j] = PHASE == 0 || d0 + j >= D ? 0.f : (single ? n_slot[(long)2 * blockIdx.z * H * D + d] : n_mine[d]);
        }
    }

    // Loads are asked for 16 rows ahead of their use (the raw numbers of the rows prepared next, the values of the rows
    // used next) and moved to the registers that are read before the following ones are asked for: no wait between two
    // barriers meets a load that was just issued.  They have no branches: rows beyond the chunk read its last one again,
    // channels beyond the head its last four; what is read there is not used.
    RecRaw raw[NPT], raw_next[NPT];
    float vv[4], v_next[4], gate_next[4] = {0.f, 0.f, 0.f, 0.f}, gate_held[4], fl[4], fl_next[4];
    float rowf = 1.f, rows_k = 0.f, rowf_next = 1.f, rows_k_next = 0.f;          // (SCALAR: the decay and the key's factor of the lane's row)
    const TA* qc = q + (long)row0 * a.row_stride + (long)hk * D;
    const TA* kc = k + (long)row0 * a.row_stride + (long)hk * D;
    const TA* vc = v + (long)row0 * a.row_stride + (long)h * Dv + (col_ok ? col : 0);
    const float* wc = MODE == 1 || MODE == 3 ? a.wx + (long)row0 * a.w_stride + (long)h * D : nullptr;
    const long row_scalar = (long)row0 * a.w_stride + h * a.w_head;
    const int stride = (int)a.row_stride, w_stride = (int)a.w_stride;
    auto fetch = [&](int base) {
        const int row = min(base + r, n - 1);
        if (SCALAR) {
            rowf_next = a.wx[row_scalar + (long)row * w_stride];
            rows_k_next = a.ks[row_scalar + (long)row * w_stride];
        }
#pragma unroll
        for (int p = 0; p < NPT; ++p) {
            const int d = min((wave + p * waves) * 16 + 4 * g, D - 4);
            if (PHASE == 1) load4(qc + row * stride + d, raw_next[p].q);
            load4(kc + row * stride + d, raw_next[p].k);
            if (MODE == 1 || MODE == 3) load4(wc + row * w_stride + d, raw_next[p].w);
        }
    };
    auto shift = [](float (&x)[4], int by) {               // x[j] <- x[j + by] where there is one
        const float y[4] = {x[0], x[1], x[2], x[3]};
#pragma unroll
        for (int j = 0; j < 4; ++j) x[j] = by == 0 ? y[j] : (by == 1 ? y[j < 3 ? j + 1 : 3] : (by == 2 ? y[j < 2 ? j + 2 : 3] : y[3]));
    };
    auto take = [&]() {
        if (SCALAR) { rowf = rowf_next; rows_k = rows_k_next; }
#pragma unroll
        for (int p = 0; p < NPT; ++p) {
            raw[p] = raw_next[p];
            if (D % 4) {                                   // (the head's last channels were read from its last four)
                const int d0 = (wave + p * waves) * 16 + 4 * g, by = d0 > D - 4 ? min(d0 - (D - 4), 3) : 0;
                if (PHASE == 1) shift(raw[p].q, by);
                shift(raw[p].k, by);
                if (MODE == 1 || MODE == 3) shift(raw[p].w, by);
            }
        }
    };
    auto fetch_values = [&](int base) {
#pragma unroll
        for (int j = 0; j < 4; ++j) v_next[j] = Elem<TA>::load(vc + min(base + 4 * g + j, n - 1) * stride);
        if (DIV && PHASE == 1) {
#pragma unroll
            for (int j = 0; j < 4; ++j) fl_next[j] = a.fl[row_scalar + (long)min(base + 4 * g + j, n - 1) * w_stride];
        }
    };
    auto fetch_gates = [&](int base) {                     // (asked for when the rows are used, read when they are written, a round later)
        if (PHASE == 1 && a.gate) {
#pragma unroll
            for (int j = 0; j < 4; ++j)
                gate_next[j] = rec_gate(a, row0 + min(base + 4 * g + j, n - 1), h * Dv + (col_ok ? col : 0));
        }
    };
    auto take_values = [&](int base) {
#pragma unroll
        for (int j = 0; j < 4; ++j) {
            const float x = (a.act_silu && MODE != 2) ? silu_quick(v_next[j]) : v_next[j];
            vv[j] = col_ok && base + 4 * g + j < n ? x : 0.f;
            if (DIV && PHASE == 1) fl[j] = fl_next[j];
            if (PHASE == 1) gate_held[j] = gate_next[j];
        }
    };
    auto prepare = [&](int base, int buf) {
        const int nb = n - base < 16 ? n - base : 16;
        const int qb = PHASE == 1 ? buf : 0;
        floatx4 ga = {0.f, 0.f, 0.f, 0.f};
        if constexpr (SCALAR) {
            if (wave >= DT) return;                        // (the same for the whole wave)
            const float f = r < nb ? rowf : 1.f;
            float F = f, B = 1.f, tot = f;
            auto scan = [&](auto half) {
                constexpr int hh = decltype(half)::value;
                const bool second = (r & hh) != 0;
                const float o = other_half<hh>(tot);
                F *= second ? o : 1.f;
                B *= second ? 1.f : o;
                tot *= o;
            };
            scan(std::integral_constant<int, 1>{});
            scan(std::integral_constant<int, 2>{});
            scan(std::integral_constant<int, 4>{});
            scan(std::integral_constant<int, 8>{});
            float M[4] = {1.f, 1.f, 1.f, 1.f};             // the product of the decays after row r up to row 4 g + i; 0 before row r
            if (PHASE == 1) {
                float run = 1.f;
#pragma unroll
                for (int u = 1; u < 16; ++u) {
                    const float fu = __builtin_bit_cast(float, __builtin_amdgcn_readlane(__builtin_bit_cast(int, f), u));
                    run = u > r ? run * fu : 1.f;
                    M[u & 3] = g == (u >> 2) ? run : M[u & 3];
                }
#pragma unroll
                for (int i = 0; i < 4; ++i) M[i] = 4 * g + i >= r ? M[i] : 0.f;
            }
            float dn = 0.f;
#pragma unroll
            for (int p = 0; p < NPT; ++p) {
                const int ct = wave + p * waves;
                if (ct >= DT) break;
                const int d0 = ct * 16 + 4 * g;
                floatx4 wq, wk, wg, qv;
#pragma unroll
                for (int j = 0; j < 4; ++j) {
                    const bool in = r < nb && d0 + j < D;
                    float kv = a.act_silu ? silu_quick(raw[p].k[j]) : raw[p].k[j];
                    kv = in ? kv * rows_k : 0.f;
                    qv[j] = 0.f;
                    if (PHASE == 1) {
                        const float x = a.act_silu ? silu_quick(raw[p].q[j]) : raw[p].q[j];
                        qv[j] = in ? x * a.q_scale : 0.f;
                    }
                    wk[j] = kv;
                }
                if (PHASE == 1) {
                    floatx4 t = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
                    for (int j = 0; j < 4; ++j) t = __builtin_amdgcn_mfma_f32_16x16x4f32(qv[j], wk[j], t, 0, 0, 0);
#pragma unroll
                    for (int i = 0; i < 4; ++i) ga[i] = fmaf(t[i], M[i], ga[i]);
                }
#pragma unroll
                for (int j = 0; j < 4; ++j) {
                    wq[j] = qv[j] * F;
                    wk[j] *= B;
                    wg[j] = tot;
                    whole[p][j] *= tot;
                    if (DIV) {
                        dn = fmaf(wq[j], nn[p][j], dn);
                        nn[p][j] = fmaf(tot, nn[p][j], row16_sum(wk[j]));
                    }
                }
                if (PHASE == 1) *(floatx4*)&qt[qb][r][d0] = wq;
                *(floatx4*)&kt[buf][r][d0] = wk;
                if (r == 0) *(floatx4*)&gt[buf][d0] = wg;
            }
            if (PHASE == 1) {
#pragma unroll
                for (int i = 0; i < 4; ++i) at[qb][wave][4 * g + i][r] = ga[i];
                if (DIV) {
                    float x, y;
                    pair_across_rows(dn, x, y);
                    dn = x + y;
                    pair_across_halves(dn, x, y);
                    dn = x + y;
                    if (g == 0) dnt[qb][wave][0][r] = dn;
#pragma unroll
                    for (int i = 0; i < 4; ++i) {
                        const float all = row16_sum(ga[i]);
                        if (r == 0) dnt[qb][wave][1][4 * g + i] = all;
                    }
                }
            }
            return;
        }
#pragma unroll
        for (int p = 0; p < NPT; ++p) {
            const int ct = wave + p * waves;
            if (ct >= DT) break;                           // (the same for the whole wave)
            const int d0 = ct * 16 + 4 * g;
            float qv[4], kv[4], F[4], B[4], tot[4];
#pragma unroll
            for (int j = 0; j < 4; ++j) {
                const bool in = r < nb && d0 + j < D;
                float f = 1.f;
                qv[j] = kv[j] = 0.f;
                if (PHASE == 1) qv[j] = (a.act_silu ? silu_quick(raw[p].q[j]) : raw[p].q[j]) * a.q_scale;
                if (MODE == 2) {
                    forget_gate(raw[p].k[j] + bias[p][j], low[p][j], f, kv[j]);
                } else {
                    kv[j] = a.act_silu ? silu_quick(raw[p].k[j]) : raw[p].k[j];
                    f = MODE == 0 ? dec : (MODE == 3 ? raw[p].w[j] : expf(-expf(raw[p].w[j] + bias[p][j])));
                }
                qv[j] = in ? qv[j] : 0.f;                  // (what lies beyond the rows and channels changes nothing)
                kv[j] = in ? kv[j] : 0.f;
                f = in ? f : 1.f;
                F[j] = MODE == 1 ? 1.f : f;
                B[j] = 1.f;
                tot[j] = f;
            }
            if (PHASE == 1) {                              // the diagonal: row r's own key
                float dg = 0.f;
#pragma unroll
                for (int j = 0; j < 4; ++j) dg = fmaf(MODE == 1 ? qv[j] * low[p][j] : qv[j], kv[j], dg);
                float x, y;
                pair_across_rows(dg, x, y);
                dg = x + y;
                pair_across_halves(dg, x, y);
                dg = x + y;
#pragma unroll
                for (int i = 0; i < 4; ++i) ga[i] += (4 * g + i == r) ? dg : 0.f;
            }
            auto level = [&](auto half) {
                constexpr int hh = decltype(half)::value;
                const bool second = (r & hh) != 0;
                if (PHASE == 1) {
                    floatx4 t = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
                    for (int j = 0; j < 4; ++j) {
                        const float x = second ? qv[j] * F[j] : kv[j] * B[j];
                        t = __builtin_amdgcn_mfma_f32_16x16x4f32(x, x, t, 0, 0, 0);
                    }
#pragma unroll
                    for (int i = 0; i < 4; ++i) {          // row 4 g + i of the second half, column r of the first half of its block
                        const int row = 4 * g + i;
                        ga[i] += ((row & hh) != 0 && !second && (row & ~(2 * hh - 1)) == (r & ~(2 * hh - 1))) ? t[i] : 0.f;
                    }
                }
#pragma unroll
                for (int j = 0; j < 4; ++j) {
                    const float o = other_half<hh>(tot[j]);
                    F[j] *= second ? o : 1.f;
                    B[j] *= second ? 1.f : o;
                    tot[j] *= o;
                }
            };
            level(std::integral_constant<int, 1>{});
            level(std::integral_constant<int, 2>{});
            level(std::integral_constant<int, 4>{});
            level(std::integral_constant<int, 8>{});
            floatx4 wq, wk, wg;
#pragma unroll
            for (int j = 0; j < 4; ++j) {
                wq[j] = qv[j] * F[j];
                wk[j] = kv[j] * B[j];
                wg[j] = tot[j];
                whole[p][j] *= tot[j];
            }
            if (PHASE == 1) *(floatx4*)&qt[qb][r][d0] = wq;
            *(floatx4*)&kt[buf][r][d0] = wk;
            if (r == 0) *(floatx4*)&gt[buf][d0] = wg;
        }
        if (PHASE == 1 && wave < PREP) {
#pragma unroll
            for (int i = 0; i < 4; ++i) at[qb][wave][4 * g + i][r] = ga[i];
        }
    };
    const int out_stride = H * Dv;
    const long out0 = (long)row0 * out_stride + (long)h * Dv + col;
    if (PHASE == 1)
        for (int i = threadIdx.x; i < 2 * W * 16; i += blockDim.x) (&sq[0][0][0])[i] = 0.f;      // (waves without columns leave no sums)
    floatx4 o_held = {0.f, 0.f, 0.f, 0.f};                 // (with a norm: the outputs of the last 16 rows)
    auto use = [&](int base, int buf) {
        const int nb = n - base < 16 ? n - base : 16;
        const int qb = PHASE == 1 ? buf : 0;
        if (PHASE == 1) {
            floatx4 av = {0.f, 0.f, 0.f, 0.f}, o = {0.f, 0.f, 0.f, 0.f}, o2 = {0.f, 0.f, 0.f, 0.f};   // (two chains)
#pragma unroll
            for (int w = 0; w < PREP; ++w) av += *(const floatx4*)&at[qb][w][r][4 * g];
#pragma unroll
            for (int ct = 0; ct < DT; ++ct) {
                const floatx4 x = *(const floatx4*)&qt[qb][r][ct * 16 + 4 * g];
#pragma unroll
                for (int j = 0; j < 4; ++j) {
                    if (ct & 1) o2 = __builtin_amdgcn_mfma_f32_16x16x4f32(x[j], S[ct][j], o2, 0, 0, 0);
                    else o = __builtin_amdgcn_mfma_f32_16x16x4f32(x[j], S[ct][j], o, 0, 0, 0);
                }
            }
#pragma unroll
            for (int j = 0; j < 4; ++j) o = __builtin_amdgcn_mfma_f32_16x16x4f32(av[j], vv[j], o, 0, 0, 0);
            o += o2;
            if (DIV) {
                floatx4 dn = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
                for (int w = 0; w < PREP; ++w) dn += *(const floatx4*)&dnt[qb][w][0][4 * g] + *(const floatx4*)&dnt[qb][w][1][4 * g];
#pragma unroll
                for (int i = 0; i < 4; ++i) o[i] /= fmaxf(fabsf(dn[i]), fl[i]) + 1e-6f;
            }
            if (a.norm_w) {
                o_held = o;
#pragma unroll
                for (int i = 0; i < 4; ++i) {              // (columns beyond the head's are zeros)
                    const float q2 = row16_sum(o[i] * o[i]);
                    if (r == 0) sq[qb][wave][4 * g + i] = q2;
                }
            } else {
#pragma unroll
                for (int i = 0; i < 4; ++i)
                    if (col_ok && 4 * g + i < nb) a.out[out0 + (base + 4 * g + i) * out_stride] = o[i];
            }
        }
#pragma unroll
        for (int ct = 0; ct < DT; ++ct) {
            S[ct] *= *(const floatx4*)&gt[buf][ct * 16 + 4 * g];
#pragma unroll
            for (int j = 0; j < 4; ++j)
                S[ct] = __builtin_amdgcn_mfma_f32_16x16x4f32(kt[buf][4 * g + j][ct * 16 + r], vv[j], S[ct], 0, 0, 0);
        }
    };
    const float inv_dv = 1.f / (float)Dv;
    const float nw = PHASE == 1 && a.norm_w && col_ok ? a.norm_w[h * Dv + col] : 0.f;
    auto write_normed = [&](int base, int buf, const float (&gates)[4]) {           // rows whose squares' sums the last barrier has made whole
        const int nb = n - base < 16 ? n - base : 16;
        const int qb = PHASE == 1 ? buf : 0;
        floatx4 all = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int w = 0; w < W; ++w) all += *(const floatx4*)&sq[qb][w][4 * g];
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            float x = o_held[i] * rsqrtf(fmaf(all[i], inv_dv, a.norm_eps)) * nw;
            if (a.gate) {
                const float p = __builtin_amdgcn_rcpf(1.f + __expf(-gates[i]));
                x *= a.gate_act == 1 ? gates[i] * p : p;
            }
            if (col_ok && 4 * g + i < nb) rec_store(a, row0 + base + 4 * g + i, h * Dv + col, x * a.y_scale);
        }
    };
    const bool prepares_first = W == 8 ? (wave & 4) == 0 : (blockIdx.y & 1) == 0;
    fetch(0);
    take();
    fetch(16);
    fetch_values(0);
    prepare(0, 0);
    __syncthreads();
#pragma unroll 1
    for (int base = 0, buf = 0; base < n; base += 16, buf ^= 1) {
        const bool more = base + 16 < n;
        take();
        take_values(base);
        __builtin_amdgcn_sched_barrier(0);
        fetch(base + 32);
        fetch_values(base + 16);
        fetch_gates(base);
        __builtin_amdgcn_sched_barrier(0);
        if (PHASE == 1 && a.norm_w && base > 0 && has_cols) write_normed(base - 16, buf ^ 1, gate_held);
        if (more && prepares_first) prepare(base + 16, buf ^ 1);
        if (has_cols) use(base, buf);
        if (more && !prepares_first) prepare(base + 16, buf ^ 1);
        __syncthreads();
    }
    if (PHASE == 1 && a.norm_w && has_cols) write_normed((n - 1) / 16 * 16, ((n - 1) / 16) & 1, gate_next);
    if (PHASE == 0 || single) {
        float* to = PHASE == 0 ? mine : slot;
#pragma unroll
        for (int ct = 0; ct < DT; ++ct)
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                const int d = ct * 16 + 4 * g + i;
                if (col_ok && d < D) to[(long)d * Dv + col] = S[ct][i];
            }
    }
    if (PHASE == 0 && blockIdx.z == 0 && r == 0) {
#pragma unroll
        for (int p = 0; p < NPT; ++p)
#pragma unroll
            for (int j = 0; j < 4; ++j) {
                const int d = (wave + p * waves) * 16 + 4 * g + j;
                if (wave + p * waves < DT && d < D) {
                    rec_ws_g(a)[((long)c * H + h) * D + d] = whole[p][j];
                    if (DIV) n_mine[d] = nn[p][j];
                }
            }
    }
    if (DIV && PHASE == 1 && single && r == 0) {           // the copies of n that belong to this block's columns
        const int copies = rec_copies(Dv);
#pragma unroll
        for (int p = 0; p < NPT; ++p)
#pragma unroll
            for (int j = 0; j < 4; ++j) {
                const int d = (wave + p * waves) * 16 + 4 * g + j;
                if (wave + p * waves < DT && d < D)
                    for (int z = 2 * blockIdx.z; z < min(2 * (int)blockIdx.z + 2, copies); ++z) n_slot[(long)z * H * D + d] = nn[p][j];
            }
    }
}

// grid (portions, H, blocks of 256 state numbers): S_in of every chunk replaces the chunk's contribution in ws; the
// portion's last state goes to the request's slot.  Mode 5: numbers D * Dv .. are n's.
static __global__ __launch_bounds__(256) void recurrence_scan_kernel(Rec a) {
    const int e = blockIdx.z * blockDim.x + threadIdx.x;
    const int pi = blockIdx.x, h = blockIdx.y, H = a.H, D = a.D, Dv = a.Dv;
    const int c0 = a.portions[3 * pi], nc = a.portions[3 * pi + 1];
    const bool is_n = e >= D * Dv;
    if (nc <= 1 || e >= D * Dv + (a.mode == 5 ? D : 0)) return;      // (a portion of one chunk reads and writes its slot itself)
    const int d = is_n ? e - D * Dv : e / Dv;
    float* slot = a.state + (long)a.tok_seq[a.portions[3 * pi + 2]] * a.state_stride;
    float* sp = is_n ? slot + (long)H * D * Dv + (long)h * D + d : slot + (long)h * D * Dv + e;
    float* ws = is_n ? rec_ws_n(a) + (long)h * D + d : a.ws + (long)h * D * Dv + e;
    const float* ws_g = rec_ws_g(a) + (long)h * D + d;
    const long step = (long)H * D * (is_n ? 1 : Dv), step_g = (long)H * D;      // from chunk to chunk
    float S = *sp;
    constexpr int N = 8;                                   // chunks asked for at a time
    for (int c = c0; c < c0 + nc; c += N) {
        float add[N], dec[N];
#pragma unroll
        for (int i = 0; i < N; ++i) {
            const long at = c + i < c0 + nc ? c + i : c0 + nc - 1;
            add[i] = ws[at * step];
            dec[i] = ws_g[at * step_g];
        }
#pragma unroll
        for (int i = 0; i < N; ++i)
            if (c + i < c0 + nc) {
                ws[(c + i) * step] = S;
                S = fmaf(dec[i], S, add[i]);
            }
    }
    *sp = S;
    if (is_n)
        for (int z = 1; z < rec_copies(Dv); ++z) sp[(long)z * H * D] = S;
}

template <typename TA, int MODE, int PHASE>
static int launch_chunks(const Rec& a, hipStream_t stream) {
    const int tiles = (a.D + 15) / 16, vt = a.Dv >= 128 ? 8 : (a.Dv + 15) / 16;
#define QE_RC(DT_)                                                                                                   \
    if (tiles <= DT_) {                                                                                              \
        int waves = DT_ > vt ? DT_ : vt;                                                                             \
        if (waves > 8) waves = 8;                                                                                    \
        recurrence_chunks_kernel<TA, MODE, PHASE, DT_, 8><<<dim3(a.n_chunks, a.H, (a.Dv + 127) / 128), waves * 64, 0, stream>>>(a); \
        QE_LAUNCH_CHECK();                                                                                           \
        return 0;                                                                                                    \
    }
    QE_RC(2) QE_RC(4)
    // Heads of many key channels and few value columns: only as many waves as have columns, each preparing two tiles of
    // channels, so that several blocks share a compute unit and none of their waves prepares only.
    if constexpr (MODE >= 3) {
        if (vt <= 4 && tiles <= 8) {
            recurrence_chunks_kernel<TA, MODE, PHASE, 8, 4><<<dim3(a.n_chunks, a.H, 1), 256, 0, stream>>>(a);
            QE_LAUNCH_CHECK();
            return 0;
        }
    }
    QE_RC(6) QE_RC(8) QE_RC(16)
#undef QE_RC
    qe_set_error("linear_recurrence: heads of %d key channels (at most 256)", a.D);
    return -1;
}

template <typename TA, int MODE>
static int launch_phases(const Rec& a, hipStream_t stream) {
    if (!a.all_single) {
        const int rc = launch_chunks<TA, MODE, 0>(a, stream);
        if (rc) return rc;
        const int numbers = a.D * a.Dv + (MODE == 5 ? a.D : 0);
        recurrence_scan_kernel<<<dim3(a.n_portions, a.H, (numbers + 255) / 256), 256, 0, stream>>>(a);
        QE_LAUNCH_CHECK();
    }
    return launch_chunks<TA, MODE, 1>(a, stream);
}
