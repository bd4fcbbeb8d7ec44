// Mixers that carry a matrix per head from token to token instead of keys and values:
//
//   qe_token_shift        n blends of every row with the row of the token before it in its request,
//                         y_s = x + (x' - x) * mu_s; what lies before a request's rows in this step comes from
//                         its state row (zeros for a new request), which then takes the request's last row
//   qe_linear_recurrence  per head, with a state S [D][Dv] in 32-bit, the recurrences listed at Rec
//                         (recurrence_gates.h): one decay a head, a decay per key channel, a forget gate that also decides
//                         what is written, decays formed beforehand per channel or per row and head, a normaliser beside S
//   qe_recurrence_single  the same for rows that are each the only row of their request, the norm per head and the gate inside
//   qe_gated_norm         y = o / rms(o) * weight * act(gate) * scale, the root mean square over each of
//                         `groups` equal pieces of a row (one: the whole row)
//
// Rows of a request are consecutive in the flat batch and tok_seq[t] names the request's state row, so a
// request's rows are found from tok_seq alone: the block of a request's first row walks on until tok_seq
// changes, every other block leaves at once.  Launch grids follow the number of rows alone.
// Everything is summed token by token in one fixed order: results do not depend on how a request was cut
// into steps or on what else is in the batch.  The recurrences' arithmetic is 32-bit throughout.
#include "recurrence_gates.h"

// ---- blends with the token before ---------------------------------------------------------------------
// grid (T); mode 0: read the state, write y; mode 1: the rows that are their request's last write the state;
// mode 2: both (the caller knows that no two rows belong to one request)
template <typename TA>
__global__ void token_shift_kernel(const TA* __restrict__ x, const float* __restrict__ mu, int n,
                                   float* __restrict__ state, long state_stride, const int* __restrict__ tok_seq,
                                   TA* __restrict__ y, int T, int W, int mode) {
    const long t = blockIdx.x;
    const int seq = tok_seq[t];
    float* st = state + (long)seq * state_stride;
    if (mode == 1) {
        if (t + 1 < T && tok_seq[t + 1] == seq) return;
        for (int c = threadIdx.x; c < W; c += blockDim.x) st[c] = Elem<TA>::load(x + t * W + c);
        return;
    }
    const bool from_state = mode == 2 || t == 0 || tok_seq[t - 1] != seq;
    for (int c = threadIdx.x; c < W; c += blockDim.x) {
        const float h = Elem<TA>::load(x + t * W + c);
        const float hp = from_state ? st[c] : Elem<TA>::load(x + (t - 1) * W + c);
        for (int s = 0; s < n; ++s)
            Elem<TA>::store(y + ((long)s * T + t) * W + c, fmaf(hp - h, mu[s * W + c], h));
        if (mode == 2) st[c] = h;
    }
}

extern "C" int qe_token_shift(const void* x, const float* mu, int n, float* state, long state_stride,
                              const int* tok_seq, void* y, int T, int W, int single_rows, int dt_a,
                              hipStream_t stream) {
    QE_REQUIRE(T >= 0 && W > 0 && n > 0 && state_stride >= W, "token_shift: bad sizes");
    if (T == 0) return 0;
    const int threads = W >= 1024 ? 256 : (W >= 256 ? 128 : 64);
#define QE_TS(TA_, mode_) token_shift_kernel<TA_><<<T, threads, 0, stream>>>((const TA_*)x, mu, n, state, state_stride, tok_seq, (TA_*)y, T, W, mode_)
    if (dt_a == QE_F32) { if (single_rows) QE_TS(float, 2); else { QE_TS(float, 0); QE_TS(float, 1); } }
    else if (dt_a == QE_BF16) { if (single_rows) QE_TS(bf16_t, 2); else { QE_TS(bf16_t, 0); QE_TS(bf16_t, 1); } }
    else QE_REQUIRE(false, "token_shift: unknown element type %d", dt_a);
#undef QE_TS
    QE_LAUNCH_CHECK();
    return 0;
}

// ---- the recurrences -----------------------------------------------------------------------------------
// A block = one request's rows of this step x one head x up to 64 value columns.  Thread (dg, v): value column
// v, key channels dg * DPG .. dg * DPG + DPG - 1 of the state in registers (REC_DG groups share a column).  Tokens
// are taken REC_TB at a time: their q, k and decays go through shared memory once (activations and the decay's
// exponentials are applied there, once per token and channel), every thread adds its channels' share of the
// outputs token by token, and the groups' shares are added in the order of the groups at the end of the batch.
#define REC_TB 16
#define REC_DG 4

template <typename TA, int DPG, int MODE>
__global__ __launch_bounds__(REC_DG * 64) void linear_recurrence_kernel(Rec a) {
    const int t0 = blockIdx.x;
    const int* __restrict__ tok_seq = a.tok_seq;
    const int seq = tok_seq[t0];
    if (t0 > 0 && tok_seq[t0 - 1] == seq) return;          // not a request's first row (the whole block leaves)
    const int T = a.T, H = a.H, D = a.D, Dv = a.Dv;
    const int h = blockIdx.y, hk = h / (H / a.Hk);
    const int tid = threadIdx.x, vl = tid & 63, dg = tid >> 6;
    const int col = blockIdx.z * 64 + vl;
    const bool col_ok = col < Dv;
    const int d0 = dg * DPG;
    const TA* __restrict__ q = (const TA*)a.q + (long)hk * D;
    const TA* __restrict__ k = (const TA*)a.k + (long)hk * D;
    const TA* __restrict__ v = (const TA*)a.v + (long)h * Dv;
    constexpr int DP = DPG * REC_DG;                        // channels with the padding
    __shared__ float sq[REC_TB][DP], sk[REC_TB][DP], sw[REC_TB][DP];
    __shared__ float part[REC_TB][REC_DG][64];
    __shared__ float den[MODE == 5 ? REC_TB : 1][REC_DG];

    float S[DPG], uu[DPG], nn[MODE == 5 ? DPG : 1];
    float* slot = a.state + (long)seq * a.state_stride;
    float* Sp = slot + ((long)h * D) * Dv + col;
    float* np = slot + (long)H * D * Dv + ((long)blockIdx.z * H + h) * D;        // (mode 5: this block's copy of n)
#pragma unroll
    for (int i = 0; i < DPG; ++i) {
        const int d = d0 + i;
        S[i] = (col_ok && d < D) ? Sp[(long)d * Dv] : 0.f;
        uu[i] = (MODE == 1 && d < D) ? a.u[h * D + d] : 0.f;
        if (MODE == 5) nn[i] = d < D ? np[d] : 0.f;
    }
    const float dec = MODE == 0 ? a.decay[h] : 0.f;

    int tb = t0;
    bool more = true;
    while (more) {
        // the batch's rows: tb .. tb + nb - 1, as far as they are this request's
        int nb = 0;
        while (nb < REC_TB && tb + nb < T && tok_seq[tb + nb] == seq) ++nb;
        more = nb == REC_TB && tb + nb < T && tok_seq[tb + nb] == seq;
        __syncthreads();                                     // (the batch before has been read)
        for (int i = tid; i < nb * DP; i += REC_DG * 64) {
            const int tt = i / DP, d = i - tt * DP;
            float x = 0.f, y = 0.f, c = 0.f;
            if (d < D) {
                const long r = (long)(tb + tt) * a.row_stride + d, wr = (long)(tb + tt) * a.w_stride;
                x = Elem<TA>::load(q + r);
                y = Elem<TA>::load(k + r);
                if (a.act_silu) { x = silu_f(x); if (MODE != 2) y = silu_f(y); }
                x *= a.q_scale;
                if (MODE == 2) { const float z = y + a.w0[h * D + d]; forget_gate(z, a.u[h * D + d], c, y); }
                if (MODE == 1) c = expf(-expf(a.wx[wr + h * D + d] + a.w0[h * D + d]));
                if (MODE == 3) c = a.wx[wr + h * D + d];
                if (MODE >= 4) { c = a.wx[wr + h * a.w_head]; y *= a.ks[wr + h * a.w_head]; }
            }
            sq[tt][d] = x; sk[tt][d] = y; sw[tt][d] = c;
        }
        float vv[REC_TB];
#pragma unroll
        for (int tt = 0; tt < REC_TB; ++tt) {
            vv[tt] = 0.f;
            if (tt < nb && col_ok) {
                vv[tt] = Elem<TA>::load(v + (long)(tb + tt) * a.row_stride + col);
                if (a.act_silu && MODE != 2) vv[tt] = silu_f(vv[tt]);
            }
        }
        __syncthreads();
#pragma unroll
        for (int tt = 0; tt < REC_TB; ++tt) {
            float o = 0.f, dn = 0.f;
            if (tt < nb) {
                const float vt = vv[tt];
#pragma unroll
                for (int i = 0; i < DPG; ++i) {
                    const float kv = sk[tt][d0 + i] * vt;
                    if (MODE == 0) {
                        S[i] = fmaf(dec, S[i], kv);
                        o = fmaf(sq[tt][d0 + i], S[i], o);
                    } else if (MODE == 1) {
                        o = fmaf(sq[tt][d0 + i], fmaf(uu[i], kv, S[i]), o);
                        S[i] = fmaf(sw[tt][d0 + i], S[i], kv);
                    } else {
                        S[i] = fmaf(sw[tt][d0 + i], S[i], kv);
                        o = fmaf(sq[tt][d0 + i], S[i], o);
                    }
                    if (MODE == 5) {
                        nn[i] = fmaf(sw[tt][d0 + i], nn[i], sk[tt][d0 + i]);
                        dn = fmaf(sq[tt][d0 + i], nn[i], dn);
                    }
                }
            }
            part[tt][dg][vl] = o;
            if (MODE == 5 && vl == 0) den[tt][dg] = dn;
        }
        __syncthreads();
        for (int i = tid; i < nb * 64; i += REC_DG * 64) {
            const int tt = i >> 6, c = i & 63;
            if (blockIdx.z * 64 + c < Dv) {
                float o = part[tt][0][c];
#pragma unroll
                for (int g = 1; g < REC_DG; ++g) o += part[tt][g][c];
                if (MODE == 5) {
                    float dn = den[tt][0];
#pragma unroll
                    for (int g = 1; g < REC_DG; ++g) dn += den[tt][g];
                    o /= fmaxf(fabsf(dn), a.fl[(long)(tb + tt) * a.w_stride + h * a.w_head]) + 1e-6f;
                }
                a.out[((long)(tb + tt) * H + h) * Dv + blockIdx.z * 64 + c] = o;
            }
        }
        tb += nb;
    }
#pragma unroll
    for (int i = 0; i < DPG; ++i) {
        const int d = d0 + i;
        if (col_ok && d < D) Sp[(long)d * Dv] = S[i];
        if (MODE == 5 && vl == 0 && d < D) np[d] = nn[i];
    }
}

// Row by row; out float32 [T, H, Dv] (norm_w is not looked at).
extern "C" int qe_linear_recurrence(const Rec* rec, hipStream_t stream) {
    const Rec& a = *rec;
    QE_REC_CHECK(a, "linear_recurrence", false);
    QE_REQUIRE(a.out, "linear_recurrence: no place for the outputs");
    if (a.T == 0) return 0;
    dim3 grid(a.T, a.H, rec_copies(a.Dv));
    const int dpg = a.D <= 32 ? 8 : (a.D <= 64 ? 16 : (a.D <= 128 ? 32 : 64));
#define QE_LR3(TA_, DPG_, MODE_) linear_recurrence_kernel<TA_, DPG_, MODE_><<<grid, REC_DG * 64, 0, stream>>>(a)
#define QE_LR2(TA_, DPG_)                                                                                     \
    switch (a.mode) {                                                                                         \
        case 0: QE_LR3(TA_, DPG_, 0); break;                                                                  \
        case 1: QE_LR3(TA_, DPG_, 1); break;                                                                  \
        case 2: QE_LR3(TA_, DPG_, 2); break;                                                                  \
        case 3: QE_LR3(TA_, DPG_, 3); break;                                                                  \
        case 4: QE_LR3(TA_, DPG_, 4); break;                                                                  \
        default: QE_LR3(TA_, DPG_, 5);                                                                        \
    }
#define QE_LR(TA_) do { if (dpg == 8) QE_LR2(TA_, 8) else if (dpg == 16) QE_LR2(TA_, 16) else if (dpg == 32) QE_LR2(TA_, 32) else QE_LR2(TA_, 64) } while (0)
    if (a.dt_a == QE_F32) QE_LR(float);
    else QE_LR(bf16_t);
#undef QE_LR
#undef QE_LR2
#undef QE_LR3
    QE_LAUNCH_CHECK();
    return 0;
}

// ---- single new tokens, the norm per head and the gate behind the recurrence inside ---------------------------------
// A block per (row, head); every row is the only row of its request.  A thread holds V neighbouring value columns and
// every RG-th key channel: its state numbers are all asked for before the gates are formed, so that one trip to memory
// serves both.  The outputs' shares are added in the order of the row groups; then the head's root mean square, the
// weight, the gate and the rounding.
#define RS_THREADS 512
#define RS_HOLD 16       // state pieces a thread asks for ahead

template <typename TA, int MODE, int V>
__global__ __launch_bounds__(RS_THREADS) void recurrence_single_kernel(Rec a) {
    extern __shared__ float sm[];                            // q, k, f, bonus of D channels, then RG x Dv shares
    __shared__ float red[16], red2[16];
    const int H = a.H, D = a.D, Dv = a.Dv;
    float* sq = sm, * sk = sm + D, * sf = sm + 2 * D, * sb = sm + 3 * D, * part = sm + 4 * D;
    const long t = blockIdx.x;
    const int h = blockIdx.y, hk = h / (H / a.Hk), tid = threadIdx.x;
    const int cols = Dv / V, RG = RS_THREADS / cols;
    const int rg = tid / cols, col = (tid - rg * cols) * V;
    const bool on = rg < RG;
    float* slot = a.state + (long)a.tok_seq[t] * a.state_stride;
    float* Sp = slot + (long)h * D * Dv;
    const TA* vp = (const TA*)a.v + t * a.row_stride + (long)h * Dv;
    auto load = [&](const float* p, float (&x)[V]) {
        if constexpr (V == 4) Vec4<float>::load(p, x);
        else x[0] = *p;
    };
    auto store = [&](float* p, const float (&x)[V]) {
        if constexpr (V == 4) Vec4<float>::store(p, x);
        else *p = x[0];
    };
    float S[RS_HOLD][V];
    if (on) {
#pragma unroll
        for (int i = 0; i < RS_HOLD; ++i) load(Sp + (long)min(rg + i * RG, D - 1) * Dv + col, S[i]);
    }
    const float gate0 = a.gate && tid < Dv ? rec_gate(a, t, h * Dv + tid) : 0.f;      // (the first of a thread's columns)
    float keep = 0.f, write = 0.f, floor = 0.f, m_new = 0.f;     // (mode 5: of the row and head)
    if (MODE == 5) {
        if (a.z) {
            float i, f;
            const float m = slot[a.m_at + h];
            memory_gates_of(a.z[t * a.z_stride + h] + a.ib[h], a.z[t * a.z_stride + H + h] + a.fb[h], a.cap, i, f);
            m_new = fmaxf(f + m, i);
            keep = expf(f + m - m_new);
            write = expf(i - m_new);
            floor = expf(-m_new);
        } else {
            keep = a.wx[t * a.w_stride + h * a.w_head];
            write = a.ks[t * a.w_stride + h * a.w_head];
            floor = a.fl[t * a.w_stride + h * a.w_head];
        }
    }
    for (int d = tid; d < D; d += RS_THREADS) {
        const long at = t * a.row_stride + (long)hk * D + d;
        float x = Elem<TA>::load((const TA*)a.q + at), y = Elem<TA>::load((const TA*)a.k + at), f = 0.f;
        if (a.act_silu) { x = silu_f(x); if (MODE != 2) y = silu_f(y); }
        x *= a.q_scale;
        if (MODE == 0) f = a.decay[h];
        if (MODE == 1) f = expf(-expf(a.wx[t * a.w_stride + h * D + d] + a.w0[h * D + d]));
        if (MODE == 2) { const float z = y + a.w0[h * D + d]; forget_gate(z, a.u[h * D + d], f, y); }
        if (MODE == 3) {
            if (a.low) {
                float z = a.b2[h * D + d];
                constexpr int N = 16;                        // asked for at a time (beyond the rank: its last again, unused)
                for (int r0 = 0; r0 < a.rank; r0 += N) {
                    float w[N], l[N];
#pragma unroll
                    for (int j = 0; j < N; ++j) {
                        const int r = min(r0 + j, a.rank - 1);
                        const long i = t * a.low_stride + r;
                        w[j] = a.w2[(long)r * H * D + h * D + d];
                        l[j] = a.dt_low == QE_F32 ? ((const float*)a.low)[i] : bf16_to_float(((const bf16_t*)a.low)[i]);
                    }
#pragma unroll
                    for (int j = 0; j < N; ++j)
                        if (r0 + j < a.rank) z = fmaf(w[j], l[j], z);
                }
                f = low_rank_decay(z, a.inv_tau);
            } else {
                f = a.wx[t * a.w_stride + h * D + d];
            }
        }
        if (MODE == 4) { f = a.wx[t * a.w_stride + h * a.w_head]; y *= a.ks[t * a.w_stride + h * a.w_head]; }
        if (MODE == 5) { f = keep; y *= write; }
        sq[d] = x; sk[d] = y; sf[d] = f;
        if (MODE == 1) sb[d] = a.u[h * D + d];
    }
    float dn = 0.f;
    if (MODE == 5) {                                         // (a thread's own channels: no barrier needed)
        const float* np = slot + (long)H * D * Dv + (long)h * D;
        for (int d = tid; d < D; d += RS_THREADS) {
            const float n = fmaf(sf[d], np[d], sk[d]);
            dn = fmaf(sq[d], n, dn);
            sb[d] = n;
        }
    }
    float vv[V], o[V];
#pragma unroll
    for (int e = 0; e < V; ++e) {
        o[e] = 0.f;
        vv[e] = 0.f;
        if (on) {
            vv[e] = Elem<TA>::load(vp + col + e);
            if (a.act_silu && MODE != 2) vv[e] = silu_f(vv[e]);
        }
    }
    __syncthreads();
    auto channel = [&](int d, float (&x)[V]) {
#pragma unroll
        for (int e = 0; e < V; ++e) {
            const float kv = sk[d] * vv[e];
            if (MODE == 1) {
                o[e] = fmaf(sq[d], fmaf(sb[d], kv, x[e]), o[e]);
                x[e] = fmaf(sf[d], x[e], kv);
            } else {
                x[e] = fmaf(sf[d], x[e], kv);
                o[e] = fmaf(sq[d], x[e], o[e]);
            }
        }
        store(Sp + (long)d * Dv + col, x);
    };
    if (on) {
#pragma unroll
        for (int i = 0; i < RS_HOLD; ++i)
            if (rg + i * RG < D) channel(rg + i * RG, S[i]);
        for (int d = rg + RS_HOLD * RG; d < D; d += RG) {
            float x[V];
            load(Sp + (long)d * Dv + col, x);
            channel(d, x);
        }
        store(part + rg * Dv + col, o);
    }
    float inv = 1.f;
    if (MODE == 5) {
        const int copies = rec_copies(Dv);
        for (int d = tid; d < D; d += RS_THREADS)
            for (int z = 0; z < copies; ++z) slot[(long)H * D * Dv + ((long)z * H + h) * D + d] = sb[d];
        dn = block_sum(dn, red2);
        inv = 1.f / (fmaxf(fabsf(dn), floor) + 1e-6f);
        if (a.z && tid == 0) slot[a.m_at + h] = m_new;       // (behind barriers that everyone reached after reading it)
    }
    __syncthreads();
    float all = 0.f;
    for (int c = tid; c < Dv; c += RS_THREADS) {
        float x = 0.f;
        for (int i = 0; i < RG; ++i) x += part[i * Dv + c];
        if (MODE == 5) x *= inv;
        part[c] = x;                                         // (this thread alone reads and writes column c)
        all = fmaf(x, x, all);
    }
    if (!a.norm_w) {
        for (int c = tid; c < Dv; c += RS_THREADS) a.out[(t * H + h) * Dv + c] = part[c];
        return;
    }
    const float rs = rsqrtf(block_sum(all, red) / (float)Dv + a.norm_eps) * a.y_scale;
    for (int c = tid; c < Dv; c += RS_THREADS) {
        float x = part[c] * rs * a.norm_w[h * Dv + c];
        if (a.gate) x *= gate_value(c == tid ? gate0 : rec_gate(a, t, h * Dv + c), a.gate_act);
        rec_store(a, t, h * Dv + c, x);
    }
}

extern "C" int qe_recurrence_single_supported(int D, int Dv) {
    return D > 0 && D <= 256 && Dv > 0 && (Dv % 4 == 0 ? Dv / 4 : Dv) <= RS_THREADS;
}

// As qe_linear_recurrence for rows that are each the only row of their request; with norm_w the norm and the gate too.
extern "C" int qe_recurrence_single(const Rec* rec, hipStream_t stream) {
    const Rec& a = *rec;
    QE_REC_CHECK(a, "recurrence_single", true);
    QE_REQUIRE(qe_recurrence_single_supported(a.D, a.Dv), "recurrence_single: heads of %d x %d", a.D, a.Dv);
    QE_REQUIRE(a.norm_w || a.out, "recurrence_single: no place for the outputs");
    if (a.T == 0) return 0;
    const bool four = a.Dv % 4 == 0 && a.state_stride % 4 == 0 && (((unsigned long)a.state) & 15) == 0;
    QE_REQUIRE(four || a.Dv <= RS_THREADS, "recurrence_single: heads of %d x %d", a.D, a.Dv);
    const int cols = four ? a.Dv / 4 : a.Dv, RG = RS_THREADS / cols;
    const size_t lds = (size_t)(4 * a.D + RG * a.Dv) * sizeof(float);
#define QE_RS4(TA_, M_, V_) recurrence_single_kernel<TA_, M_, V_><<<dim3(a.T, a.H), RS_THREADS, lds, stream>>>(a)
#define QE_RS3(TA_, M_) do { if (four) QE_RS4(TA_, M_, 4); else QE_RS4(TA_, M_, 1); } while (0)
#define QE_RS(TA_)                                  \
    switch (a.mode) {                               \
        case 0: QE_RS3(TA_, 0); break;              \
        case 1: QE_RS3(TA_, 1); break;              \
        case 2: QE_RS3(TA_, 2); break;              \
        case 3: QE_RS3(TA_, 3); break;              \
        case 4: QE_RS3(TA_, 4); break;              \
        default: QE_RS3(TA_, 5);                    \
    }
    if (a.dt_a == QE_F32) QE_RS(float)
    else QE_RS(bf16_t)
#undef QE_RS
#undef QE_RS3
#undef QE_RS4
    QE_LAUNCH_CHECK();
    return 0;
}

// ---- norm, gate --------------------------------------------------------------------------------------
// One block per row, a wave per group in turn; fewer groups than waves: all waves share every group's sums through
// shared memory.  gate_act: 0 none, 1 silu, 2 sigmoid.
template <typename TG, typename TO>
__global__ void gated_norm_kernel(const float* __restrict__ o, const float* __restrict__ weight,
                                  const TG* __restrict__ gate, long gate_stride, int gate_act, float eps, float scale,
                                  TO* __restrict__ y, long y_stride, int N, int groups) {
    const long t = blockIdx.x;
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, nw = blockDim.x >> 6;
    const int n = N / groups;
    if (groups < nw) {
        __shared__ float part[16];
        for (int g = 0; g < groups; ++g) {
            const float* og = o + t * N + (long)g * n;
            float a = 0.f;
            for (int c = threadIdx.x; c < n; c += blockDim.x) a += og[c] * og[c];
            a = wave_sum(a);
            __syncthreads();                                 // (the group before has been read)
            if (lane == 0) part[wave] = a;
            __syncthreads();
            float all = 0.f;
            for (int w = 0; w < nw; ++w) all += part[w];     // (every thread adds in the order of the waves)
            const float f = rsqrtf(all / (float)n + eps);
            for (int c = threadIdx.x; c < n; c += blockDim.x) {
                const int cc = g * n + c;
                float val = og[c] * f * weight[cc];
                if (gate) {
                    const float z = Elem<TG>::load(gate + t * gate_stride + cc);
                    val *= gate_act == 1 ? silu_f(z) : (gate_act == 2 ? sigmoid_f(z) : z);
                }
                Elem<TO>::store(y + t * y_stride + cc, val * scale);
            }
        }
        return;
    }
    for (int g = wave; g < groups; g += nw) {
        const float* og = o + t * N + (long)g * n;
        float a = 0.f;
        for (int c = lane; c < n; c += 64) a += og[c] * og[c];
        a = wave_sum(a);
        const float f = rsqrtf(a / (float)n + eps);
        for (int c = lane; c < n; c += 64) {
            const int cc = g * n + c;
            float val = og[c] * f * weight[cc];
            if (gate) {
                const float z = Elem<TG>::load(gate + t * gate_stride + cc);
                val *= gate_act == 1 ? silu_f(z) : (gate_act == 2 ? sigmoid_f(z) : z);
            }
            Elem<TO>::store(y + t * y_stride + cc, val * scale);
        }
    }
}

extern "C" int qe_gated_norm(const float* o, const float* weight, const void* gate, long gate_stride, int dt_g,
                             int gate_act, float eps, float scale, void* y, long y_stride, int dt_y, int T, int N,
                             int groups, hipStream_t stream) {
    QE_REQUIRE(T >= 0 && N > 0 && groups > 0 && N % groups == 0, "gated_norm: rows of %d in %d groups", N, groups);
    QE_REQUIRE(y_stride >= N && (!gate || gate_stride >= N), "gated_norm: rows overlap");
    if (T == 0) return 0;
    const int threads = (groups >= 4 || N / groups >= 512) ? 256 : 64 * groups;   // (long groups: four waves share each)
#define QE_GN(TG_, TO_) gated_norm_kernel<TG_, TO_><<<T, threads, 0, stream>>>(o, weight, (const TG_*)gate, gate_stride, gate_act, eps, scale, (TO_*)y, y_stride, N, groups)
    const int dg = gate ? dt_g : dt_y;
    if (dg == QE_F32 && dt_y == QE_F32) QE_GN(float, float);
    else if (dg == QE_BF16 && dt_y == QE_BF16) QE_GN(bf16_t, bf16_t);
    else if (dg == QE_F32 && dt_y == QE_BF16) QE_GN(float, bf16_t);
    else QE_REQUIRE(false, "gated_norm: no kernel for gate type %d with output type %d", dt_g, dt_y);
#undef QE_GN
    QE_LAUNCH_CHECK();
    return 0;
}

// ---- activations between two products, and what is done to the logits ------------------------------------
// kind 0: exact gelu, 0.5 z (1 + erf(z / sqrt 2)); 1: tanh; 2: cap * tanh(z / cap); 3: a * x + b * y
template <typename TI, typename TO>
__global__ void unary_kernel(const TI* __restrict__ z, TO* __restrict__ y, long n, int kind, float cap) {
    const long i = (long)blockIdx.x * blockDim.x + threadIdx.x;
    if (i >= n) return;
    const float v = Elem<TI>::load(z + i);
    float r;
    if (kind == 0) r = 0.5f * v * (1.f + erff(v * 0.70710678118654752440f));
    else if (kind == 1) r = tanhf(v);
    else r = cap * tanhf(v / cap);
    Elem<TO>::store(y + i, r);
}

extern "C" int qe_unary(const void* z, int dt_z, void* y, int dt_y, long n, int kind, float cap, hipStream_t stream) {
    QE_REQUIRE(n >= 0 && kind >= 0 && kind <= 2, "unary: bad arguments");
    if (n == 0) return 0;
    const int blocks = qe_cdiv(n, 256);
    if (dt_z == QE_F32 && dt_y == QE_F32) unary_kernel<float, float><<<blocks, 256, 0, stream>>>((const float*)z, (float*)y, n, kind, cap);
    else if (dt_z == QE_F32 && dt_y == QE_BF16) unary_kernel<float, bf16_t><<<blocks, 256, 0, stream>>>((const float*)z, (bf16_t*)y, n, kind, cap);
    else if (dt_z == QE_BF16 && dt_y == QE_BF16) unary_kernel<bf16_t, bf16_t><<<blocks, 256, 0, stream>>>((const bf16_t*)z, (bf16_t*)y, n, kind, cap);
    else QE_REQUIRE(false, "unary: no kernel from type %d to type %d", dt_z, dt_y);
    QE_LAUNCH_CHECK();
    return 0;
}

template <typename TI>
__global__ void scaled_sum_kernel(const TI* __restrict__ a, float sa, const TI* __restrict__ b, float sb,
                                  float* __restrict__ y, long n) {
    const long i = (long)blockIdx.x * blockDim.x + threadIdx.x;
    if (i < n) y[i] = fmaf(sb, Elem<TI>::load(b + i), sa * Elem<TI>::load(a + i));
}

extern "C" int qe_scaled_sum(const void* a, float sa, const void* b, float sb, int dt, float* y, long n,
                             hipStream_t stream) {
    QE_REQUIRE(n >= 0, "scaled_sum: bad size");
    if (n == 0) return 0;
    const int blocks = qe_cdiv(n, 256);
    if (dt == QE_F32) scaled_sum_kernel<float><<<blocks, 256, 0, stream>>>((const float*)a, sa, (const float*)b, sb, y, n);
    else if (dt == QE_BF16) scaled_sum_kernel<bf16_t><<<blocks, 256, 0, stream>>>((const bf16_t*)a, sa, (const bf16_t*)b, sb, y, n);
    else QE_REQUIRE(false, "scaled_sum: unknown element type %d", dt);
    QE_LAUNCH_CHECK();
    return 0;
}
