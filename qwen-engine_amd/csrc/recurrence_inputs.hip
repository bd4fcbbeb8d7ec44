// What the recurrences whose decays are formed beforehand (recurrence_gates.h, modes 3 to 5) read beside their q, k and v, and
// what stands behind one of them.  All 32-bit but the convolved rows, which are activations.
//
//   qe_memory_gates      per head, from the logits of an input and a forget gate: i = cap * tanh(z_i / cap), log f = log
//                        sigmoid(cap * tanh(z_f / cap)), the running maximum m_t = max(log f + m_(t-1), i) and from it the
//                        decay exp(log f + m_(t-1) - m_t), the key's factor exp(i - m_t) and the floor exp(-m_t)
//   qe_low_rank_decay    sigmoid(W low + b)^(1 / tau) per channel, low a few numbers a row
//   qe_conv_steps        a causal convolution over time on each channel with a bias, then silu; beside it the step sizes
//                        dt = softplus(z + bias) and the decays exp(-exp(A) dt)
//   qe_skip_gate_norm    y = (o + D_h x) * silu(z), normed in equal groups of a row, times a weight
#include "recurrence_gates.h"

// ---- the gates of a matrix memory ------------------------------------------------------------------------------------
struct MemoryGates {
    const float* z;              // [T] rows: H input gates, H forget gates; parts of them z_part apart, to be added in order
    long z_stride, z_part;
    int parts;
    const float* ib;
    const float* fb;
    float cap;
    float* state;                // m of head h at + slot * state_stride + h
    long state_stride;
    const int* tok_seq;
    float* out;                  // decay, key factor, floor of row t and head h at + k * o_kind + t * o_row + h * o_head
    long o_kind, o_row, o_head;
    int T, H;
    const int* chunks;           // of the chunked recurrence, or null
    const int* portions;
};
__device__ __forceinline__ void memory_gates_at(const MemoryGates& a, long t, int h, float& i, float& f) {
    const float* z = a.z + t * a.z_stride + h;
    float zi = z[0], zf = z[a.H];
    for (int p = 1; p < a.parts; ++p) { zi += z[p * a.z_part]; zf += z[p * a.z_part + a.H]; }
    memory_gates_of(zi + a.ib[h], zf + a.fb[h], a.cap, i, f);
}

// grid (T): the block of a request's first row walks its rows, a thread a head
__global__ __launch_bounds__(64) void memory_gates_rows_kernel(MemoryGates a) {
    const int t0 = blockIdx.x, seq = a.tok_seq[t0];
    if (t0 > 0 && a.tok_seq[t0 - 1] == seq) return;
    for (int h = threadIdx.x; h < a.H; h += blockDim.x) {
        float* ms = a.state + (long)seq * a.state_stride + h;
        float m = *ms, i, f;
        for (int t = t0; t < a.T && a.tok_seq[t] == seq; ++t) {
            memory_gates_at(a, t, h, i, f);
            const float n = fmaxf(f + m, i);
            float* o = a.out + t * a.o_row + h * a.o_head;
            o[0] = expf(f + m - n);
            o[a.o_kind] = expf(i - n);
            o[2 * a.o_kind] = expf(-n);
            m = n;
        }
        *ms = m;
    }
}

// Many rows: every gate first (log f in the decay's place, i in the key factor's), a thread a row and head ...
__global__ __launch_bounds__(256) void memory_gates_each_kernel(MemoryGates a) {
    const int n = blockIdx.x * 256 + threadIdx.x, t = n / a.H, h = n - t * a.H;
    if (t >= a.T) return;
    float i, f;
    memory_gates_at(a, t, h, i, f);
    float* o = a.out + t * a.o_row + h * a.o_head;
    o[0] = f;
    o[a.o_kind] = i;
}

// ... then the running maximum: grid (portions, H), MG_ROWS neighbouring rows a thread, MG_THREADS of them at a time.  The
// maximum over what lies before a thread's rows is a scan over pairs (sum of log f, maximum), (F1, M1) then (F2, M2) being
// (F1 + F2, max(M1 + F2, M2)): no sum is ever taken off another.
#define MG_THREADS 1024
#define MG_ROWS 2
__global__ __launch_bounds__(MG_THREADS) void memory_gates_scan_kernel(MemoryGates a) {
    __shared__ float wf[MG_THREADS / 64], wm[MG_THREADS / 64];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, h = blockIdx.y;
    const int* po = a.portions + 3 * blockIdx.x;
    const int* last = a.chunks + 3 * (po[0] + po[1] - 1);
    const long first = po[2];
    const int n = last[0] + last[1] - (int)first;
    float* out = a.out + first * a.o_row + h * a.o_head;
    float* ms = a.state + (long)a.tok_seq[first] * a.state_stride + h;
    float m0 = *ms;                                        // the running maximum before the rows of this turn
    for (int b = 0; b < n; b += MG_THREADS * MG_ROWS) {
        const int t0 = b + tid * MG_ROWS;
        float f[MG_ROWS], i[MG_ROWS], F = 0.f, M = -INFINITY;
#pragma unroll
        for (int k = 0; k < MG_ROWS; ++k) {
            const float* o = out + min(t0 + k, n - 1) * a.o_row;
            f[k] = o[0];
            i[k] = o[a.o_kind];
        }
#pragma unroll
        for (int k = 0; k < MG_ROWS; ++k)
            if (t0 + k < n) { F += f[k]; M = fmaxf(M + f[k], i[k]); }
#pragma unroll
        for (int o = 1; o < 64; o <<= 1) {                 // inclusive over the wave
            const float pf = __shfl_up(F, o, 64), pm = __shfl_up(M, o, 64);
            if (lane >= o) { M = fmaxf(pm + F, M); F += pf; }
        }
        if (lane == 63) { wf[wave] = F; wm[wave] = M; }
        float eF = __shfl_up(F, 1, 64), eM = __shfl_up(M, 1, 64);      // what lies before this thread's rows in its wave
        if (lane == 0) { eF = 0.f; eM = -INFINITY; }
        __syncthreads();
        float m = m0, all = m0;
        for (int w = 0; w < MG_THREADS / 64; ++w) {        // the waves before, then all of them
            if (w == wave) m = all;
            all = fmaxf(all + wf[w], wm[w]);
        }
        m = fmaxf(m + eF, eM);
        m0 = all;
#pragma unroll
        for (int k = 0; k < MG_ROWS; ++k)
            if (t0 + k < n) {
                const float x = fmaxf(f[k] + m, i[k]);
                float* o = out + (t0 + k) * a.o_row;
                o[0] = expf(f[k] + m - x);
                o[a.o_kind] = expf(i[k] - x);
                o[2 * a.o_kind] = expf(-x);
                m = x;
            }
        __syncthreads();                                   // (the waves' pairs have been read)
    }
    if (tid == 0) *ms = m0;
}

// out: number (k, t, h) at k * o_kind + t * o_row + h * o_head, k = decay, key factor, floor.  chunks and portions (or null,
// with n_portions 0): as in the chunked recurrence; without them the rows of a request are walked one by one.  parts > 1: z is
// that many tensors of partial products, z_part numbers apart.
extern "C" int qe_memory_gates(const float* z, long z_stride, int parts, long z_part, const float* ib, const float* fb, float cap,
                               float* state, long state_stride, const int* tok_seq, float* out, long o_kind, long o_row, long o_head,
                               int T, int H, const int* chunks, const int* portions, int n_portions, hipStream_t stream) {
    QE_REQUIRE(T >= 0 && H > 0 && H <= 65535 && cap > 0.f && parts >= 1 && z_stride >= 2L * H && state_stride >= H, "memory_gates: bad sizes");
    QE_REQUIRE((long)T * H < (1L << 31), "memory_gates: %d rows of %d heads", T, H);
    if (T == 0) return 0;
    MemoryGates a{z, z_stride, z_part, parts, ib, fb, cap, state, state_stride, tok_seq, out, o_kind, o_row, o_head, T, H, chunks, portions};
    if (n_portions > 0) {
        QE_REQUIRE(chunks && portions, "memory_gates: portions without their chunks");
        memory_gates_each_kernel<<<qe_cdiv((long)T * H, 256), 256, 0, stream>>>(a);
        QE_LAUNCH_CHECK();
        memory_gates_scan_kernel<<<dim3(n_portions, H), MG_THREADS, 0, stream>>>(a);
    } else {
        memory_gates_rows_kernel<<<T, 64, 0, stream>>>(a);
    }
    QE_LAUNCH_CHECK();
    return 0;
}

// ---- decays through a low rank ---------------------------------------------------------------------------------------
// A block takes LR_ROWS rows x 256 channels, a thread a channel; the rows' low numbers pass through shared memory.
#define LR_ROWS 8
template <typename TL>
__global__ __launch_bounds__(256) void low_rank_decay_kernel(const TL* __restrict__ low, long low_stride,
                                                             const float* __restrict__ w, const float* __restrict__ bias,
                                                             float inv_tau, float* __restrict__ out, int T, int N, int R) {
    extern __shared__ float ls[];                          // [R][LR_ROWS]
    const int t0 = blockIdx.x * LR_ROWS, c = blockIdx.y * 256 + threadIdx.x, cc = min(c, N - 1);
    constexpr int AHEAD = 16;                              // weights asked for before the rows' numbers are waited for
    float wv[AHEAD];
#pragma unroll
    for (int j = 0; j < AHEAD; ++j) wv[j] = w[(long)min(j, R - 1) * N + cc];
    const float b = bias[cc];
    for (int i = threadIdx.x; i < LR_ROWS * R; i += 256) {
        const int tt = i / R, r = i - tt * R;
        ls[r * LR_ROWS + tt] = t0 + tt < T ? Elem<TL>::load(low + (long)(t0 + tt) * low_stride + r) : 0.f;
    }
    __syncthreads();
    if (c >= N) return;
    float acc[LR_ROWS];
#pragma unroll
    for (int tt = 0; tt < LR_ROWS; ++tt) acc[tt] = b;
    for (int r0 = 0; r0 < R; r0 += AHEAD) {
        if (r0 > 0) {
#pragma unroll
            for (int j = 0; j < AHEAD; ++j) wv[j] = w[(long)min(r0 + j, R - 1) * N + c];
        }
#pragma unroll
        for (int j = 0; j < AHEAD; ++j)
            if (r0 + j < R) {
#pragma unroll
                for (int tt = 0; tt < LR_ROWS; ++tt) acc[tt] = fmaf(wv[j], ls[(r0 + j) * LR_ROWS + tt], acc[tt]);
            }
    }
#pragma unroll
    for (int tt = 0; tt < LR_ROWS; ++tt)
        if (t0 + tt < T) out[(long)(t0 + tt) * N + c] = low_rank_decay(acc[tt], inv_tau);
}

// low [T] rows of R numbers (dt_l), w [R][N], bias [N] -> out float32 [T][N]
extern "C" int qe_low_rank_decay(const void* low, long low_stride, int dt_l, const float* w, const float* bias, float tau,
                                 float* out, int T, int N, int R, hipStream_t stream) {
    QE_REQUIRE(T >= 0 && N > 0 && R > 0 && R <= 1024 && tau > 0.f && low_stride >= R, "low_rank_decay: bad sizes (rank %d)", R);
    if (T == 0) return 0;
    const dim3 grid(qe_cdiv(T, LR_ROWS), qe_cdiv(N, 256));
    const size_t lds = (size_t)R * LR_ROWS * sizeof(float);
    if (dt_l == QE_F32) low_rank_decay_kernel<float><<<grid, 256, lds, stream>>>((const float*)low, low_stride, w, bias, 1.f / tau, out, T, N, R);
    else if (dt_l == QE_BF16) low_rank_decay_kernel<bf16_t><<<grid, 256, lds, stream>>>((const bf16_t*)low, low_stride, w, bias, 1.f / tau, out, T, N, R);
    else QE_REQUIRE(false, "low_rank_decay: unknown element type %d", dt_l);
    QE_LAUNCH_CHECK();
    return 0;
}

// ---- convolution over time with bias and silu, step sizes and decays ---------------------------------------------------
// The inputs before a request's rows of this step are its state [taps - 1][C] in 32-bit (zeros at the start), brought up to
// date with its last inputs: by the same launch where every row is the only row of its request, else by one behind it.
struct ConvSteps {
    const void* x;               // [T] rows of C numbers, x_stride apart
    long x_stride;
    const float* w;              // [taps][C]
    const float* b;              // [C]
    float* state;
    long state_stride;
    const int* tok_seq;
    void* out;                   // [T][C]
    int T, C, taps;
    const float* dt;             // [T] rows of H numbers, or null; parts of them dt_part apart, to be added in order
    long dt_stride, dt_part;
    int dt_parts;
    const float* dt_bias;
    const float* A_log;
    float* steps;                // [T][2 H]: decays, dt
    int H;
    int single;
};
#define CS_ROWS 8

__device__ __forceinline__ void conv_step_sizes(const ConvSteps& a, long t, int h) {
    float z = a.dt[t * a.dt_stride + h];
    for (int p = 1; p < a.dt_parts; ++p) z += a.dt[p * a.dt_part + t * a.dt_stride + h];
    z += a.dt_bias[h];
    const float dt = fmaxf(z, 0.f) + log1pf(expf(-fabsf(z)));
    a.steps[t * 2 * a.H + h] = expf(-expf(a.A_log[h]) * dt);
    a.steps[t * 2 * a.H + a.H + h] = dt;
}

// A thread walks CS_ROWS rows (single: one) of V channels and keeps the inputs before its row in registers.  The last
// column of blocks forms the step sizes.
template <typename TA, int TAPS, int V>
__global__ __launch_bounds__(256) void conv_steps_kernel(ConvSteps a, int col_blocks) {
    constexpr int N1 = TAPS - 1;
    const int rows = a.single ? 1 : CS_ROWS, t0 = blockIdx.y * rows;
    if ((int)blockIdx.x == col_blocks) {
        for (int i = threadIdx.x; i < rows * a.H; i += 256) {
            const int tt = i / a.H;
            if (t0 + tt < a.T) conv_step_sizes(a, t0 + tt, i - tt * a.H);
        }
        return;
    }
    const int c = (blockIdx.x * 256 + threadIdx.x) * V;
    if (c >= a.C) return;
    const TA* x = (const TA*)a.x + c;
    TA* out = (TA*)a.out + c;
    auto load = [&](long t, float (&v)[V]) {
        if constexpr (V == 4) Vec4<TA>::load(x + t * a.x_stride, v);
        else v[0] = Elem<TA>::load(x + t * a.x_stride);
    };
    auto load_f = [&](const float* p, float (&v)[V]) {
        if constexpr (V == 4) Vec4<float>::load(p, v);
        else v[0] = *p;
    };
    float w[TAPS][V], bias[V], hist[N1 > 0 ? N1 : 1][V];   // hist[k]: the input k + 1 rows back
#pragma unroll
    for (int k = 0; k < TAPS; ++k) load_f(a.w + (long)k * a.C + c, w[k]);
    load_f(a.b + c, bias);
    int s = -1;
    for (int tt = 0; tt < rows; ++tt) {
        const long t = t0 + tt;
        if (t >= a.T) break;
        const int seq = a.tok_seq[t];
        if (N1 > 0 && (tt == 0 || seq != s)) {             // a request's rows begin, or this thread's
            const float* st = a.state + (long)seq * a.state_stride + c;
            int before = 0;
            if (tt == 0 && !a.single)
                while (before < N1 && t - 1 - before >= 0 && a.tok_seq[t - 1 - before] == seq) ++before;
#pragma unroll
            for (int k = 0; k < N1; ++k) {
                if (k < before) load(t - 1 - k, hist[k]);
                else load_f(st + (long)(N1 - 1 - k + before) * a.C, hist[k]);
            }
        }
        s = seq;
        float xt[V], y[V];
        load(t, xt);
#pragma unroll
        for (int e = 0; e < V; ++e) {
            float v = bias[e];
#pragma unroll
            for (int k = N1; k >= 1; --k) v = fmaf(w[TAPS - 1 - k][e], hist[k - 1][e], v);   // the oldest input first
            v = fmaf(w[TAPS - 1][e], xt[e], v);
            y[e] = silu_f(v);
        }
        if constexpr (V == 4) Vec4<TA>::store(out + t * a.C, y);
        else Elem<TA>::store(out + t * a.C, y[0]);
#pragma unroll
        for (int k = N1 - 1; k >= 1; --k)
#pragma unroll
            for (int e = 0; e < V; ++e) hist[k][e] = hist[k - 1][e];
        if (N1 > 0) {
#pragma unroll
            for (int e = 0; e < V; ++e) hist[0][e] = xt[e];
        }
    }
    if (N1 > 0 && a.single) {
        float* st = a.state + (long)s * a.state_stride + c;
#pragma unroll
        for (int k = 0; k < N1; ++k) {
            if constexpr (V == 4) Vec4<float>::store(st + (long)(N1 - 1 - k) * a.C, hist[k]);
            else st[(long)(N1 - 1 - k) * a.C] = hist[k][0];
        }
    }
}

// Any number of taps, a thread a row and channel.
template <typename TA>
__global__ __launch_bounds__(256) void conv_steps_any_kernel(ConvSteps a, int col_blocks) {
    const long t = blockIdx.y;
    if ((int)blockIdx.x == col_blocks) {
        for (int h = threadIdx.x; h < a.H; h += 256) conv_step_sizes(a, t, h);
        return;
    }
    const int c = blockIdx.x * 256 + threadIdx.x;
    if (c >= a.C) return;
    const int n1 = a.taps - 1, seq = a.tok_seq[t];
    const TA* x = (const TA*)a.x + c;
    float* st = a.state + (long)seq * a.state_stride + c;
    int before = 0;
    if (!a.single)
        while (before < n1 && t - 1 - before >= 0 && a.tok_seq[t - 1 - before] == seq) ++before;
    float v = a.b[c];
    for (int k = n1; k >= 0; --k) {
        const float in = k <= before ? Elem<TA>::load(x + (t - k) * a.x_stride) : st[(long)(n1 - k + before) * a.C];
        v = fmaf(a.w[(long)(n1 - k) * a.C + c], in, v);
        if (a.single && k < n1) st[(long)(n1 - 1 - k) * a.C] = in;
    }
    Elem<TA>::store((TA*)a.out + t * a.C + c, silu_f(v));
}

// A request's last inputs into its state.  With portions: grid y = portions; else grid y = rows, the last row of a request
// working.
template <typename TA>
__global__ __launch_bounds__(256) void conv_steps_state_kernel(ConvSteps a, const int* chunks, const int* portions) {
    const int c = blockIdx.x * 256 + threadIdx.x;
    if (c >= a.C) return;
    const int n1 = a.taps - 1;
    long first, end;
    if (portions) {
        const int* po = portions + 3 * blockIdx.y;
        const int* last = chunks + 3 * (po[0] + po[1] - 1);
        first = po[2];
        end = last[0] + last[1];
    } else {
        const long t = blockIdx.y;
        if (t + 1 < a.T && a.tok_seq[t + 1] == a.tok_seq[t]) return;
        end = t + 1;
        first = t;
        while (end - first < n1 && first > 0 && a.tok_seq[first - 1] == a.tok_seq[t]) --first;
    }
    float* st = a.state + (long)a.tok_seq[first] * a.state_stride + c;
    const TA* x = (const TA*)a.x + c;
    const long n = end - first;
    for (int j = 0; j < n1; ++j) {                         // (ascending: an entry is read before it is written over)
        const long t = end - n1 + j;
        st[(long)j * a.C] = t >= first ? Elem<TA>::load(x + t * a.x_stride) : st[(j + n) * (long)a.C];
    }
}

// w [taps][C], b [C], state rows of (taps - 1) * C numbers; dt (or null): [T] rows of H logits -> steps [T][2 H].
extern "C" int qe_conv_steps(const void* x, long x_stride, const float* w, const float* b, float* state, long state_stride,
                             const int* tok_seq, void* out, int T, int C, int taps, const float* dt, long dt_stride,
                             int dt_parts, long dt_part, const float* dt_bias, const float* A_log, float* steps, int H, int single_rows,
                             const int* chunks, const int* portions, int n_portions, int dt_a, hipStream_t stream) {
    QE_REQUIRE(T >= 0 && C > 0 && taps >= 1 && x_stride >= C, "conv_steps: bad sizes T=%d C=%d taps=%d", T, C, taps);
    QE_REQUIRE(taps == 1 || (state && state_stride >= (long)(taps - 1) * C), "conv_steps: %d taps need a state", taps);
    QE_REQUIRE(!dt || (H > 0 && dt_bias && A_log && steps && dt_stride >= H), "conv_steps: step sizes lack operands");
    QE_REQUIRE(dt_a == QE_F32 || dt_a == QE_BF16, "conv_steps: unknown element type %d", dt_a);
    QE_REQUIRE(n_portions == 0 || (chunks && portions), "conv_steps: portions without their chunks");
    if (T == 0) return 0;
    ConvSteps a{x, x_stride, w, b, state, state_stride, tok_seq, out, T, C, taps, dt, dt_stride, dt_part, dt_parts, dt_bias, A_log, steps, H, single_rows};
    const size_t esz = dt_a == QE_BF16 ? 2 : 4;
    const bool four = C % 4 == 0 && x_stride % 4 == 0 && (((unsigned long)x) & (4 * esz - 1)) == 0 && state_stride % 4 == 0 &&
                      (((unsigned long)state) & 15) == 0;
    const int V = four ? 4 : 1;
    const int col_blocks = taps <= 4 ? qe_cdiv(C, 256 * V) : qe_cdiv(C, 256);
    const int row_blocks = taps <= 4 && !single_rows ? qe_cdiv(T, CS_ROWS) : T;
    QE_REQUIRE(row_blocks <= 65535 && T <= 65535, "conv_steps: more than 65535 rows in a step");
    const dim3 grid(col_blocks + (dt ? 1 : 0), row_blocks);
#define QE_CS(TA_, TAPS_) do { if (four) conv_steps_kernel<TA_, TAPS_, 4><<<grid, 256, 0, stream>>>(a, col_blocks);   \
                               else conv_steps_kernel<TA_, TAPS_, 1><<<grid, 256, 0, stream>>>(a, col_blocks); } while (0)
#define QE_CST(TA_)                                                                                        \
    do {                                                                                                   \
        if (taps == 1) QE_CS(TA_, 1);                                                                      \
        else if (taps == 2) QE_CS(TA_, 2);                                                                 \
        else if (taps == 3) QE_CS(TA_, 3);                                                                 \
        else if (taps == 4) QE_CS(TA_, 4);                                                                 \
        else conv_steps_any_kernel<TA_><<<grid, 256, 0, stream>>>(a, col_blocks);                          \
    } while (0)
    if (dt_a == QE_F32) QE_CST(float);
    else QE_CST(bf16_t);
#undef QE_CST
#undef QE_CS
    QE_LAUNCH_CHECK();
    if (!single_rows && taps > 1) {
        const dim3 ugrid(qe_cdiv(C, 256), n_portions > 0 ? n_portions : T);
        const int* po = n_portions > 0 ? portions : nullptr;
        if (dt_a == QE_F32) conv_steps_state_kernel<float><<<ugrid, 256, 0, stream>>>(a, chunks, po);
        else conv_steps_state_kernel<bf16_t><<<ugrid, 256, 0, stream>>>(a, chunks, po);
        QE_LAUNCH_CHECK();
    }
    return 0;
}

// ---- skip, gate, norm ------------------------------------------------------------------------------------------------
struct SkipGateNorm {
    const float* o;              // [T][N]
    const void* x;               // [T] rows, x_stride apart
    long x_stride;
    const float* skip;           // [H], head h of N / H numbers
    const void* z;               // [T] rows, z_stride apart
    long z_stride;
    const float* w;              // [N]
    float eps;
    void* y;                     // [T] rows, y_stride apart
    long y_stride;
    int N, Dv, groups;
};
template <typename TA>
__device__ __forceinline__ float skip_gate_at(const SkipGateNorm& a, long t, int c) {
    const float v = fmaf(a.skip[c / a.Dv], Elem<TA>::load((const TA*)a.x + t * a.x_stride + c), a.o[t * a.N + c]);
    return v * silu_f(Elem<TA>::load((const TA*)a.z + t * a.z_stride + c));
}

// Any sizes: a block a row, group after group, the numbers formed twice.
template <typename TA, typename TO>
__global__ __launch_bounds__(256) void skip_gate_norm_kernel(SkipGateNorm a) {
    __shared__ float red[16];
    const long t = blockIdx.x;
    const int n = a.N / a.groups;
    for (int g = 0; g < a.groups; ++g) {
        float ss = 0.f;
        for (int c = g * n + threadIdx.x; c < (g + 1) * n; c += blockDim.x) {
            const float v = skip_gate_at<TA>(a, t, c);
            ss += v * v;
        }
        const float f = rsqrtf(block_sum(ss, red) / (float)n + a.eps);
        for (int c = g * n + threadIdx.x; c < (g + 1) * n; c += blockDim.x)
            Elem<TO>::store((TO*)a.y + t * a.y_stride + c, skip_gate_at<TA>(a, t, c) * f * a.w[c]);
    }
}

// Rows of up to NV * 1024 numbers in pieces of four that stay in registers; a group is the whole row or a multiple of 256
// numbers, so that a wave's piece lies in one group.
template <typename TA, typename TO, int NV>
__global__ __launch_bounds__(256) void skip_gate_norm_regs_kernel(SkipGateNorm a) {
    __shared__ float part[NV * 4];
    const long t = blockIdx.x;
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, N = a.N, n = N / a.groups;
    float v[NV][4], zv[NV][4], xv[NV][4], w[NV][4];
    int cs[NV];
#pragma unroll
    for (int i = 0; i < NV; ++i) {
        const int c = (threadIdx.x + i * 256) * 4;
        cs[i] = c < N ? c : 0;
        Vec4<float>::load(a.o + t * N + cs[i], v[i]);
        Vec4<TA>::load((const TA*)a.x + t * a.x_stride + cs[i], xv[i]);
        Vec4<TA>::load((const TA*)a.z + t * a.z_stride + cs[i], zv[i]);
        Vec4<float>::load(a.w + cs[i], w[i]);
    }
#pragma unroll
    for (int i = 0; i < NV; ++i) {
        const bool ok = (threadIdx.x + i * 256) * 4 < N;
        const int h0 = cs[i] / a.Dv;
        const float s0 = a.skip[h0];
        float ss = 0.f;
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            const int c = cs[i] + e;
            const float s = c < (h0 + 1) * a.Dv ? s0 : a.skip[c / a.Dv];
            const float u = fmaf(s, xv[i][e], v[i][e]);
            v[i][e] = u * silu_f(zv[i][e]);
            ss += v[i][e] * v[i][e];
        }
        ss = wave_sum(ok ? ss : 0.f);
        if (lane == 0) part[i * 4 + wave] = ss;            // piece i * 4 + wave: numbers 256 (4 i + wave) ..
    }
    __syncthreads();
    const int per = a.groups == 1 ? NV * 4 : n / 256;
    float f_all = 0.f;
    if (a.groups == 1) {
        float all = 0.f;
        for (int p = 0; p < NV * 4; ++p) all += part[p];
        f_all = rsqrtf(all / (float)n + a.eps);
    }
#pragma unroll
    for (int i = 0; i < NV; ++i) {
        if ((threadIdx.x + i * 256) * 4 >= N) continue;
        float f = f_all;
        if (a.groups > 1) {
            const int g = (i * 4 + wave) / per;
            float all = 0.f;
            for (int p = 0; p < per; ++p) all += part[g * per + p];
            f = rsqrtf(all / (float)n + a.eps);
        }
        float o[4];
#pragma unroll
        for (int e = 0; e < 4; ++e) o[e] = v[i][e] * f * w[i][e];
        Vec4<TO>::store((TO*)a.y + t * a.y_stride + cs[i], o);
    }
}

extern "C" int qe_skip_gate_norm(const float* o, const void* x, long x_stride, const float* skip, const void* z, long z_stride,
                                 const float* w, float eps, void* y, long y_stride, int T, int H, int Dv, int groups, int dt_a, int dt_y,
                                 hipStream_t stream) {
    const int N = H * Dv;
    QE_REQUIRE(T >= 0 && H > 0 && Dv > 0 && groups > 0 && N % groups == 0, "skip_gate_norm: rows of %d in %d groups", N, groups);
    QE_REQUIRE(x_stride >= N && z_stride >= N && y_stride >= N, "skip_gate_norm: rows overlap");
    if (T == 0) return 0;
    SkipGateNorm a{o, x, x_stride, skip, z, z_stride, w, eps, y, y_stride, N, Dv, groups};
    const size_t esz = dt_a == QE_BF16 ? 2 : 4;
    const bool regs = N % 4 == 0 && N <= 8192 && (groups == 1 || (N / groups) % 256 == 0) && x_stride % 4 == 0 && z_stride % 4 == 0 && y_stride % 4 == 0 &&
                      ((((unsigned long)x) | ((unsigned long)z)) & (4 * esz - 1)) == 0 && (((unsigned long)y) & 15) == 0;
    const int nv = qe_cdiv(N, 1024);
#define QE_SGN(TA_, TO_)                                                                                     \
    do {                                                                                                     \
        if (!regs) skip_gate_norm_kernel<TA_, TO_><<<T, 256, 0, stream>>>(a);                                \
        else if (nv <= 1) skip_gate_norm_regs_kernel<TA_, TO_, 1><<<T, 256, 0, stream>>>(a);                 \
        else if (nv <= 2) skip_gate_norm_regs_kernel<TA_, TO_, 2><<<T, 256, 0, stream>>>(a);                 \
        else if (nv <= 4) skip_gate_norm_regs_kernel<TA_, TO_, 4><<<T, 256, 0, stream>>>(a);                 \
        else skip_gate_norm_regs_kernel<TA_, TO_, 8><<<T, 256, 0, stream>>>(a);                              \
    } while (0)
    if (dt_a == QE_F32 && dt_y == QE_F32) QE_SGN(float, float);
    else if (dt_a == QE_F32 && dt_y == QE_BF16) QE_SGN(float, bf16_t);
    else if (dt_a == QE_BF16 && dt_y == QE_BF16) QE_SGN(bf16_t, bf16_t);
    else QE_REQUIRE(false, "skip_gate_norm: no kernel from type %d to type %d", dt_a, dt_y);
#undef QE_SGN
    QE_LAUNCH_CHECK();
    return 0;
}
