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
#include "recurrence_gates.h"
#include <type_traits>

typedef __attribute__((ext_vector_type(4))) float floatx4;

struct RecArgs {
    const void* q;
    const void* k;
    const void* v;
    long row_stride;
    const float* wx;
    long w_stride;
    const float* w0;
    const float* u;
    const float* decay;
    int act_silu;
    const int* chunks;
    float* ws_s;                    // [chunks][H][D][Dv]
    float* ws_g;                    // [chunks][H][D]
    float* state;
    long state_stride;
    const int* tok_seq;
    float* out;                     // [T][H][Dv]; null with a norm
    int H, D, Dv;
    const float* norm_w;            // [H * Dv] or null
    float norm_eps;
    void* y;                        // [T][H * Dv] normed rows
    int y_bf16;
};

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

template <typename TA, int MODE, int PHASE, int DT>
__global__ __launch_bounds__(512) void recurrence_chunks_kernel(RecArgs a) {
    constexpr int DP = DT * 16, LD = DP + 4, NPT = (DT + 7) / 8;
    __shared__ __align__(16) float qt[PHASE == 1 ? 2 : 1][16][LD];
    __shared__ __align__(16) float kt[2][16][LD];
    __shared__ __align__(16) float gt[2][DP];
    __shared__ __align__(16) float at[PHASE == 1 ? 2 : 1][8][16][20];
    __shared__ __align__(16) float sq[PHASE == 1 ? 2 : 1][8][16];
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, waves = blockDim.x >> 6, g = lane >> 4, r = lane & 15;
    const int c = blockIdx.x, h = blockIdx.y;
    const int row0 = a.chunks[3 * c], n = a.chunks[3 * c + 1], single = a.chunks[3 * c + 2];
    if (PHASE == 0 && single) return;
    const int H = a.H, D = a.D, Dv = a.Dv;
    const int col0 = blockIdx.z * 128 + wave * 16, col = col0 + r;
    const bool has_cols = wave < 8 && col0 < Dv && wave * 16 < 128;
    const bool col_ok = has_cols && col < Dv;
    constexpr int PREP = DT < 8 ? DT : 8;                  // waves that prepare channels (the launch has at least as many)
    const TA* q = (const TA*)a.q;
    const TA* k = (const TA*)a.k;
    const TA* v = (const TA*)a.v;
    floatx4 S[DT];
    float* slot = a.state + (long)a.tok_seq[row0] * a.state_stride + (long)h * D * Dv;
    float* mine = a.ws_s + ((long)c * H + h) * D * Dv;
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
    float bias[NPT][4], low[NPT][4], whole[NPT][4];
    const float dec = MODE == 0 ? a.decay[h] : 0.f;
#pragma unroll
    for (int p = 0; p < NPT; ++p) {
        const int d0 = (wave + p * waves) * 16 + 4 * g;
#pragma unroll
        for (int j = 0; j < 4; ++j) {
            const int d = min(d0 + j, D - 1);              // (what stands beyond the head's channels is not used)
            bias[p][j] = MODE != 0 ? a.w0[h * D + d] : 0.f;
            low[p][j] = MODE != 0 ? a.u[h * D + d] : 0.f;
            whole[p][j] = 1.f;
        }
    }

    // Loads are asked for 16 rows ahead of their use (the raw numbers of the rows prepared next, the values of the rows
    // used next) and moved to the registers that are read before the following ones are asked for: no wait between two
    // barriers meets a load that was just issued.  They have no branches: rows beyond the chunk read its last one again,
    // channels beyond the head its last four; what is read there is not used.
    RecRaw raw[NPT], raw_next[NPT];
    float vv[4], v_next[4];
    const TA* qc = q + (long)row0 * a.row_stride + (long)h * D;
    const TA* kc = k + (long)row0 * a.row_stride + (long)h * D;
    const TA* vc = v + (long)row0 * a.row_stride + (long)h * Dv + (col_ok ? col : 0);
    const float* wc = MODE == 1 ? a.wx + (long)row0 * a.w_stride + (long)h * D : nullptr;
    const int stride = (int)a.row_stride, w_stride = (int)a.w_stride;
    auto fetch = [&](int base) {
        const int row = min(base + r, n - 1);
#pragma unroll
        for (int p = 0; p < NPT; ++p) {
            const int d = min((wave + p * waves) * 16 + 4 * g, D - 4);
            if (PHASE == 1) load4(qc + row * stride + d, raw_next[p].q);
            load4(kc + row * stride + d, raw_next[p].k);
            if (MODE == 1) load4(wc + row * w_stride + d, raw_next[p].w);
        }
    };
    auto shift = [](float (&x)[4], int by) {               // x[j] <- x[j + by] where there is one
        const float y[4] = {x[0], x[1], x[2], x[3]};
#pragma unroll
        for (int j = 0; j < 4; ++j) x[j] = by == 0 ? y[j] : (by == 1 ? y[j < 3 ? j + 1 : 3] : (by == 2 ? y[j < 2 ? j + 2 : 3] : y[3]));
    };
    auto take = [&]() {
#pragma unroll
        for (int p = 0; p < NPT; ++p) {
            raw[p] = raw_next[p];
            if (D % 4) {                                   // (the head's last channels were read from its last four)
                const int d0 = (wave + p * waves) * 16 + 4 * g, by = d0 > D - 4 ? min(d0 - (D - 4), 3) : 0;
                if (PHASE == 1) shift(raw[p].q, by);
                shift(raw[p].k, by);
                if (MODE == 1) shift(raw[p].w, by);
            }
        }
    };
    auto fetch_values = [&](int base) {
#pragma unroll
        for (int j = 0; j < 4; ++j) v_next[j] = Elem<TA>::load(vc + min(base + 4 * g + j, n - 1) * stride);
    };
    auto take_values = [&](int base) {
#pragma unroll
        for (int j = 0; j < 4; ++j) {
            const float x = (a.act_silu && MODE != 2) ? silu_quick(v_next[j]) : v_next[j];
            vv[j] = col_ok && base + 4 * g + j < n ? x : 0.f;
        }
    };
    auto prepare = [&](int base, int buf) {
        const int nb = n - base < 16 ? n - base : 16;
        const int qb = PHASE == 1 ? buf : 0;
        floatx4 ga = {0.f, 0.f, 0.f, 0.f};
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
                if (PHASE == 1) qv[j] = a.act_silu ? silu_quick(raw[p].q[j]) : raw[p].q[j];
                if (MODE == 2) {
                    forget_gate(raw[p].k[j] + bias[p][j], low[p][j], f, kv[j]);
                } else {
                    kv[j] = a.act_silu ? silu_quick(raw[p].k[j]) : raw[p].k[j];
                    f = MODE == 0 ? dec : expf(-expf(raw[p].w[j] + bias[p][j]));
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
        for (int i = threadIdx.x; i < 256; i += blockDim.x) (&sq[0][0][0])[i] = 0.f;      // (waves without columns leave no sums)
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
    auto write_normed = [&](int base, int buf) {           // rows whose squares' sums the last barrier has made whole
        const int nb = n - base < 16 ? n - base : 16;
        const int qb = PHASE == 1 ? buf : 0;
        floatx4 all = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int w = 0; w < 8; ++w) all += *(const floatx4*)&sq[qb][w][4 * g];
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            const float x = o_held[i] * rsqrtf(fmaf(all[i], inv_dv, a.norm_eps)) * nw;
            if (col_ok && 4 * g + i < nb) {
                const long to = out0 + (base + 4 * g + i) * out_stride;
                if (a.y_bf16) ((bf16_t*)a.y)[to] = float_to_bf16(x);
                else ((float*)a.y)[to] = x;
            }
        }
    };
    const bool prepares_first = (wave & 4) == 0;
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
        __builtin_amdgcn_sched_barrier(0);
        if (PHASE == 1 && a.norm_w && base > 0 && has_cols) write_normed(base - 16, buf ^ 1);
        if (more && prepares_first) prepare(base + 16, buf ^ 1);
        if (has_cols) use(base, buf);
        if (more && !prepares_first) prepare(base + 16, buf ^ 1);
        __syncthreads();
    }
    if (PHASE == 1 && a.norm_w && has_cols) write_normed((n - 1) / 16 * 16, ((n - 1) / 16) & 1);
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
                if (wave + p * waves < DT && d < D) a.ws_g[((long)c * H + h) * D + d] = whole[p][j];
            }
    }
}

// grid (portions, H, blocks of 256 state numbers): S_in of every chunk replaces the chunk's contribution in ws_s; the
// portion's last state goes to the request's slot
__global__ __launch_bounds__(256) void recurrence_scan_kernel(const int* __restrict__ portions, const int* __restrict__ tok_seq,
                                                              float* __restrict__ ws_s, const float* __restrict__ ws_g,
                                                              float* __restrict__ state, long state_stride, int H, int D, int Dv) {
    const int e = blockIdx.z * blockDim.x + threadIdx.x;
    const int pi = blockIdx.x, h = blockIdx.y;
    const int c0 = portions[3 * pi], nc = portions[3 * pi + 1];
    if (nc <= 1 || e >= D * Dv) return;                    // (a portion of one chunk reads and writes its slot itself)
    const int d = e / Dv, slot = tok_seq[portions[3 * pi + 2]];
    float* sp = state + (long)slot * state_stride + (long)h * D * Dv + e;
    float S = *sp;
    constexpr int N = 8;                                   // chunks asked for at a time
    for (int c = c0; c < c0 + nc; c += N) {
        float add[N], dec[N];
#pragma unroll
        for (int i = 0; i < N; ++i) {
            const long at = (long)(c + i < c0 + nc ? c + i : c0 + nc - 1) * H + h;
            add[i] = ws_s[at * D * Dv + e];
            dec[i] = ws_g[at * D + d];
        }
#pragma unroll
        for (int i = 0; i < N; ++i)
            if (c + i < c0 + nc) {
                ws_s[((long)(c + i) * H + h) * D * Dv + e] = S;
                S = fmaf(dec[i], S, add[i]);
            }
    }
    *sp = S;
}

template <typename TA, int MODE, int PHASE>
static int launch_chunks(const RecArgs& a, int n_chunks, hipStream_t stream) {
    const int tiles = (a.D + 15) / 16, vt = a.Dv >= 128 ? 8 : (a.Dv + 15) / 16;
#define QE_RC(DT_)                                                                                                   \
    if (tiles <= DT_) {                                                                                              \
        int waves = DT_ > vt ? DT_ : vt;                                                                             \
        if (waves > 8) waves = 8;                                                                                    \
        recurrence_chunks_kernel<TA, MODE, PHASE, DT_><<<dim3(n_chunks, a.H, (a.Dv + 127) / 128), waves * 64, 0, stream>>>(a); \
        QE_LAUNCH_CHECK();                                                                                           \
        return 0;                                                                                                    \
    }
    QE_RC(2) QE_RC(4) QE_RC(6) QE_RC(8) QE_RC(16)
#undef QE_RC
    qe_set_error("linear_recurrence: heads of %d key channels (at most 256)", a.D);
    return -1;
}

template <typename TA, int MODE>
static int launch_phases(const RecArgs& a, int n_chunks, const int* portions, int n_portions, int all_single, hipStream_t stream) {
    if (!all_single) {
        const int rc = launch_chunks<TA, MODE, 0>(a, n_chunks, stream);
        if (rc) return rc;
        recurrence_scan_kernel<<<dim3(n_portions, a.H, (a.D * a.Dv + 255) / 256), 256, 0, stream>>>(
            portions, a.tok_seq, a.ws_s, a.ws_g, a.state, a.state_stride, a.H, a.D, a.Dv);
        QE_LAUNCH_CHECK();
    }
    return launch_chunks<TA, MODE, 1>(a, n_chunks, stream);
}

// As qe_linear_recurrence (recurrence.hip), for rows cut into chunks on the host.  ws: float32, n_chunks * H *
// (D * Dv + D) numbers (not read if all_single: every portion is one chunk).  norm_w (float32 [H * Dv], or null; heads
// of at most 128 value columns): every head's output divided by its root mean square (norm_eps inside) and multiplied by
// the weight goes to y [T, H * Dv] in dt_y instead of out.  Rows that no chunk names are left alone.
extern "C" int qe_linear_recurrence_chunked(const void* q, const void* k, const void* v, long row_stride, const float* wx,
                                            long w_stride, const float* w0, const float* u, const float* decay, int mode,
                                            int act_silu, float* state, long state_stride, const int* tok_seq,
                                            const int* chunks, int n_chunks, const int* portions, int n_portions, int all_single,
                                            float* ws, float* out, const float* norm_w, float norm_eps, void* y, int dt_y,
                                            int H, int D, int Dv, int dt_a, hipStream_t stream) {
    QE_REQUIRE(n_chunks >= 0 && n_portions >= 0 && H > 0 && H <= 65535 && D > 0 && Dv > 0, "linear_recurrence: bad sizes");
    QE_REQUIRE(D >= 4 && D <= 256, "linear_recurrence: heads of %d key channels (4 to 256 in chunks)", D);
    QE_REQUIRE(mode == 0 ? decay != nullptr : (w0 && u && (mode == 2 || (mode == 1 && wx))), "linear_recurrence: mode %d lacks operands", mode);
    QE_REQUIRE(state_stride >= (long)H * D * Dv, "linear_recurrence: state rows overlap");
    QE_REQUIRE(dt_a == QE_F32 || dt_a == QE_BF16, "linear_recurrence: unknown element type %d", dt_a);
    if (n_chunks == 0) return 0;
    QE_REQUIRE(chunks && portions && (all_single || ws), "linear_recurrence: chunks without a workspace");
    QE_REQUIRE(row_stride < (1L << 23) && w_stride < (1L << 23) && (long)H * Dv < (1L << 23), "linear_recurrence: rows too long");
    QE_REQUIRE(norm_w ? (y && Dv <= 128 && (dt_y == QE_F32 || dt_y == QE_BF16)) : out != nullptr, "linear_recurrence: no place for the outputs, or heads too wide for the norm inside");
    RecArgs a{q, k, v, row_stride, wx, w_stride, w0, u, decay, act_silu, chunks, ws, ws + (long)n_chunks * H * D * Dv,
              state, state_stride, tok_seq, out, H, D, Dv, norm_w, norm_eps, y, dt_y == QE_BF16};
#define QE_RP(TA_) (mode == 0 ? launch_phases<TA_, 0>(a, n_chunks, portions, n_portions, all_single, stream)   \
                  : mode == 1 ? launch_phases<TA_, 1>(a, n_chunks, portions, n_portions, all_single, stream)   \
                              : launch_phases<TA_, 2>(a, n_chunks, portions, n_portions, all_single, stream))
    return dt_a == QE_F32 ? QE_RP(float) : QE_RP(bf16_t);
#undef QE_RP
}
