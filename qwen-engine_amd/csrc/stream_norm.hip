// What stands between one sublayer and the next where a layer scales its branches, averages over depth and convolves
// what its sublayers read, in as few passes over the rows as there are:
//
//   v = x + scale * (delta_0 + delta_1 + ...)          the residual sum, the branch scaled per channel (scale optional)
//   kept[k] = v                                        (optional) a layer's result, for this and later averages
//   x' = c_0 kept[0] + ... + c_(k-1) kept[k-1] + c_k v (optional) the average over depth; without it x' = v
//   h = (x' - mean) * rstd * w                         layer norm (or RMS norm: mean 0)
//   out_t = h_t + sum_j u[j] h_(t - taps + 1 + j)      (optional) causal convolution over time, zeros before the start
//
// qe_stream_norm does all of it for rows that are each the only row of their request (single new tokens: the earlier h
// come from the request's state, which is shifted in the same launch), or everything but the convolution for any rows.
// Many rows with a convolution: qe_stream_norm leaves x' and the rows' statistics, qe_norm_conv forms h from them on
// the fly (a thread walks a few consecutive rows of its channels and keeps the last taps - 1 h in registers), and a
// small kernel after it writes the requests' last taps - 1 h into their states.  All sums are 32-bit, in one fixed
// order: the parts ascending, the kept results ascending, the convolution from the oldest input on; they do not depend
// on how a request was cut into steps or on what else is in the batch.
#include "common.h"

struct StreamNorm {
    float* x;                      // [T, H]; takes x' unless rows is given
    const void* delta;             // n_delta tensors [T, H], delta_stride apart; null: none
    int n_delta;
    long delta_stride;
    const float* scale;            // [H] or null
    float* kept;                   // results, kept_stride apart; null: none
    long kept_stride;
    int k;                         // this sum's place among them
    const float* coef;             // [k + 1] or null: kept only
    const int* rows;               // the rows to norm (nothing is written back then), or null: all
    const float* w;                // norm weight
    void* out;                     // normed rows, or null
    float* stats;                  // [T][2] mean, rstd; or null
    int H;
    float eps;
    int center;
    const float* conv_w;           // [taps][H], or null: no convolution here
    float* state;                  // [slots][taps - 1][H]
    const int* tok_seq;
    int taps;
};

// One block per row, the row in registers: NV pieces of four a thread.  FEW: few rows, whose time is the latency of
// their loads: everything a row needs (the first SB parts, the first SB kept results, the weights, the convolution's taps
// and the state's rows, up to four taps) is asked for before anything is waited for, from addresses that are always valid
// (a part beyond the last reads another again and is not used); further parts and results come SB at a time.  Many rows
// are bound by the memory's rate and take two at a time.
template <typename TA, typename TD, int NV, bool FEW>
__global__ __launch_bounds__(FEW ? 512 : 256) void stream_norm_kernel(StreamNorm a) {
    constexpr int SB = !FEW ? 2 : (NV <= 1 ? 8 : (NV <= 2 ? 4 : 2));
    constexpr int ST = 3;                                  // state rows and taps asked for ahead: up to ST, ST + 1
    __shared__ float red[2][16];
    const long r = blockIdx.x;
    const long src = a.rows ? (long)a.rows[r] : r;
    const int H = a.H;
    float* xr = a.x + src * H;
    int cs[NV];
    bool ok[NV];
#pragma unroll
    for (int i = 0; i < NV; ++i) {
        const int c = (threadIdx.x + i * blockDim.x) * 4;
        ok[i] = c < H;
        cs[i] = ok[i] ? c : 0;
    }
    const int n1 = a.taps - 1;
    const bool ahead = FEW && a.conv_w && n1 <= ST;        // (the same for the whole grid, as all conditions on a's fields)
    float* st = a.conv_w ? a.state + (long)a.tok_seq[src] * n1 * H : nullptr;
    const TD* parts = (const TD*)a.delta + src * H;
    float* kr = a.kept + src * H;
    const bool averages = a.coef != nullptr && a.k > 0;

    float v[NV][4], d0[SB][NV][4], k0[SB][NV][4], c0[SB], sc[NV][4], wv[NV][4];
    float sv[FEW ? ST : 1][NV][4], uv[FEW ? ST + 1 : 1][NV][4];
    auto load_parts = [&](int s0, float (&d)[SB][NV][4]) {
#pragma unroll
        for (int s = 0; s < SB; ++s) {
            const TD* part = parts + (long)min(s0 + s, a.n_delta - 1) * a.delta_stride;
#pragma unroll
            for (int i = 0; i < NV; ++i) Vec4<TD>::load(part + cs[i], d[s][i]);
        }
    };
    auto load_kept = [&](int s0, float (&d)[SB][NV][4], float (&c)[SB]) {
#pragma unroll
        for (int s = 0; s < SB; ++s) {
            const int at = min(s0 + s, a.k - 1);
            c[s] = a.coef[at];
#pragma unroll
            for (int i = 0; i < NV; ++i) Vec4<float>::load(kr + (long)at * a.kept_stride + cs[i], d[s][i]);
        }
    };
#pragma unroll
    for (int i = 0; i < NV; ++i) Vec4<float>::load(xr + cs[i], v[i]);
    if (a.delta) load_parts(0, d0);
#pragma unroll
    for (int i = 0; i < NV; ++i) {
        sc[i][0] = sc[i][1] = sc[i][2] = sc[i][3] = 1.f;
        if (a.scale) Vec4<float>::load(a.scale + cs[i], sc[i]);
    }
    float ck = 1.f;
    if (a.coef) ck = a.coef[a.k];
    if (FEW && averages) load_kept(0, k0, c0);
    if (a.out) {
#pragma unroll
        for (int i = 0; i < NV; ++i) Vec4<float>::load(a.w + cs[i], wv[i]);
    }
    if (ahead) {
#pragma unroll
        for (int j = 0; j <= ST; ++j)
            if (j <= n1) {
#pragma unroll
                for (int i = 0; i < NV; ++i) Vec4<float>::load(a.conv_w + (long)j * H + cs[i], uv[FEW ? j : 0][i]);
            }
#pragma unroll
        for (int j = 0; j < ST; ++j)
            if (j < n1) {
#pragma unroll
                for (int i = 0; i < NV; ++i) Vec4<float>::load(st + (long)j * H + cs[i], sv[FEW ? j : 0][i]);
            }
    }
    if (a.delta) {
        float sum[NV][4] = {};
        for (int s0 = 0; s0 < a.n_delta; s0 += SB) {
            if (s0 > 0) load_parts(s0, d0);
#pragma unroll
            for (int s = 0; s < SB; ++s)
                if (s0 + s < a.n_delta) {
#pragma unroll
                    for (int i = 0; i < NV; ++i)
#pragma unroll
                        for (int e = 0; e < 4; ++e) sum[i][e] += d0[s][i][e];
                }
        }
#pragma unroll
        for (int i = 0; i < NV; ++i)
#pragma unroll
            for (int e = 0; e < 4; ++e) v[i][e] = fmaf(sc[i][e], sum[i][e], v[i][e]);
    }
    const bool write = !a.rows;
    if (a.kept) {
        if (write) {
#pragma unroll
            for (int i = 0; i < NV; ++i)
                if (ok[i]) Vec4<float>::store(kr + (long)a.k * a.kept_stride + cs[i], v[i]);
        }
        if (a.coef) {
            float acc[NV][4] = {};
            for (int s0 = 0; s0 < a.k; s0 += SB) {
                if (!FEW || s0 > 0) load_kept(s0, k0, c0);
#pragma unroll
                for (int s = 0; s < SB; ++s)
                    if (s0 + s < a.k) {
#pragma unroll
                        for (int i = 0; i < NV; ++i)
#pragma unroll
                            for (int e = 0; e < 4; ++e) acc[i][e] = fmaf(c0[s], k0[s][i][e], acc[i][e]);
                    }
            }
#pragma unroll
            for (int i = 0; i < NV; ++i)
#pragma unroll
                for (int e = 0; e < 4; ++e) v[i][e] = fmaf(ck, v[i][e], acc[i][e]);
        }
    }
    if (write && (a.delta || a.coef)) {
#pragma unroll
        for (int i = 0; i < NV; ++i)
            if (ok[i]) Vec4<float>::store(xr + cs[i], v[i]);
    }
    if (!a.out && !a.stats) return;                        // (the sums alone; the same for the whole grid)
    float mean = 0.f;
    if (a.center) {
        float sm = 0.f;
#pragma unroll
        for (int i = 0; i < NV; ++i)
            if (ok[i]) {
#pragma unroll
                for (int e = 0; e < 4; ++e) sm += v[i][e];
            }
        mean = block_sum(sm, red[0]) / (float)H;
    }
    float ss = 0.f;
#pragma unroll
    for (int i = 0; i < NV; ++i)
        if (ok[i]) {
#pragma unroll
            for (int e = 0; e < 4; ++e) ss += (v[i][e] - mean) * (v[i][e] - mean);
        }
    ss = block_sum(ss, red[1]);
    const float rstd = rsqrtf(ss / (float)H + a.eps);
    if (a.stats && threadIdx.x == 0) {
        a.stats[2 * r] = mean;
        a.stats[2 * r + 1] = rstd;
    }
    if (!a.out) return;
#pragma unroll
    for (int i = 0; i < NV; ++i) {
        if (!ok[i]) continue;
        const int c = cs[i];
        float h[4], o[4];
#pragma unroll
        for (int e = 0; e < 4; ++e) o[e] = h[e] = (v[i][e] - mean) * rstd * wv[i][e];
        if (ahead) {                                       // oldest input first
#pragma unroll
            for (int j = 0; j < ST; ++j)
                if (j < n1) {
#pragma unroll
                    for (int e = 0; e < 4; ++e) o[e] = fmaf(uv[FEW ? j : 0][i][e], sv[FEW ? j : 0][i][e], o[e]);
                    if (j > 0) Vec4<float>::store(st + (long)(j - 1) * H + c, sv[FEW ? j : 0][i]);
                }
#pragma unroll
            for (int j = 0; j <= ST; ++j)
                if (j == n1) {
#pragma unroll
                    for (int e = 0; e < 4; ++e) o[e] = fmaf(uv[FEW ? j : 0][i][e], h[e], o[e]);
                }
            if (n1 > 0) Vec4<float>::store(st + (long)(n1 - 1) * H + c, h);
        } else if (a.conv_w) {
            float u[4], p[4];
            for (int j = 0; j < n1; ++j) {
                Vec4<float>::load(st + (long)j * H + c, p);
                Vec4<float>::load(a.conv_w + (long)j * H + c, u);
#pragma unroll
                for (int e = 0; e < 4; ++e) o[e] = fmaf(u[e], p[e], o[e]);
                if (j > 0) Vec4<float>::store(st + (long)(j - 1) * H + c, p);
            }
            Vec4<float>::load(a.conv_w + (long)n1 * H + c, u);
#pragma unroll
            for (int e = 0; e < 4; ++e) o[e] = fmaf(u[e], h[e], o[e]);
            if (n1 > 0) Vec4<float>::store(st + (long)(n1 - 1) * H + c, h);
        }
        Vec4<TA>::store((TA*)a.out + r * H + c, o);
    }
}

// Any width: the row in shared memory.
template <typename TA, typename TD>
__global__ __launch_bounds__(256) void stream_norm_any_kernel(StreamNorm a) {
    extern __shared__ float row[];                         // H
    __shared__ float red[16];
    const long r = blockIdx.x;
    const long src = a.rows ? (long)a.rows[r] : r;
    const int H = a.H;
    float* xr = a.x + src * H;
    const bool write = !a.rows;
    float sm = 0.f;
    for (int c = threadIdx.x; c < H; c += blockDim.x) {
        float v = xr[c];
        if (a.delta) {
            float sum = 0.f;
            for (int s = 0; s < a.n_delta; ++s) sum += Elem<TD>::load((const TD*)a.delta + s * a.delta_stride + src * H + c);
            v = fmaf(a.scale ? a.scale[c] : 1.f, sum, v);
        }
        if (a.kept) {
            float* kr = a.kept + src * H + c;
            if (write) kr[(long)a.k * a.kept_stride] = v;
            if (a.coef) {
                float acc = 0.f;
                for (int s = 0; s < a.k; ++s) acc = fmaf(a.coef[s], kr[(long)s * a.kept_stride], acc);
                v = fmaf(a.coef[a.k], v, acc);
            }
        }
        if (write && (a.delta || a.coef)) xr[c] = v;
        row[c] = v;
        sm += v;
    }
    if (!a.out && !a.stats) return;
    const float mean = a.center ? block_sum(sm, red) / (float)H : 0.f;
    float ss = 0.f;
    for (int c = threadIdx.x; c < H; c += blockDim.x) ss += (row[c] - mean) * (row[c] - mean);   // (a thread's own entries)
    ss = block_sum(ss, red);
    const float rstd = rsqrtf(ss / (float)H + a.eps);
    if (a.stats && threadIdx.x == 0) {
        a.stats[2 * r] = mean;
        a.stats[2 * r + 1] = rstd;
    }
    if (!a.out) return;
    const int n1 = a.taps - 1;
    float* st = a.conv_w ? a.state + (long)a.tok_seq[src] * n1 * H : nullptr;
    for (int c = threadIdx.x; c < H; c += blockDim.x) {
        const float h = (row[c] - mean) * rstd * a.w[c];
        float o = h;
        if (a.conv_w) {
            for (int j = 0; j < n1; ++j) {
                const float p = st[(long)j * H + c];
                o = fmaf(a.conv_w[(long)j * H + c], p, o);
                if (j > 0) st[(long)(j - 1) * H + c] = p;
            }
            o = fmaf(a.conv_w[(long)n1 * H + c], h, o);
            if (n1 > 0) st[(long)(n1 - 1) * H + c] = h;
        }
        Elem<TA>::store((TA*)a.out + r * H + c, o);
    }
}

template <typename TA, typename TD>
static void launch_stream_norm(const StreamNorm& a, int n_rows, hipStream_t stream) {
    if (a.H % 4 == 0 && a.H <= 8192) {
        int threads = ((a.H / 4 + 63) / 64) * 64;
        const int most = n_rows <= 512 ? 512 : 256;
        if (threads > most) threads = most;
        const int nv = (a.H / 4 + threads - 1) / threads;
#define QE_SN(NV_)                                                                                  \
    do {                                                                                            \
        if (n_rows <= 512) stream_norm_kernel<TA, TD, NV_, true><<<n_rows, threads, 0, stream>>>(a); \
        else stream_norm_kernel<TA, TD, NV_, false><<<n_rows, threads, 0, stream>>>(a);             \
    } while (0)
        if (nv <= 1) QE_SN(1);
        else if (nv <= 2) QE_SN(2);
        else if (nv <= 4) QE_SN(4);
        else stream_norm_kernel<TA, TD, 8, false><<<n_rows, threads, 0, stream>>>(a);   // (few rows have at most four pieces a thread)
#undef QE_SN
        return;
    }
    stream_norm_any_kernel<TA, TD><<<n_rows, 256, (size_t)a.H * sizeof(float), stream>>>(a);
}

// dt_d: element type of delta (that of the output, or float).  conv_w [taps][H] with state and tok_seq: every row is
// the only row of its request (the caller knows).  n_rows: rows of `rows`, or T.
extern "C" int qe_stream_norm(float* x, const void* delta, int n_delta, int dt_d, const float* scale, float* kept, int k,
                              const float* coef, const int* rows, int n_rows, const float* w, void* out, float* stats,
                              int T, int H, float eps, int dt_a, int center, const float* conv_w, float* state,
                              const int* tok_seq, int taps, hipStream_t stream) {
    QE_REQUIRE(T >= 0 && n_rows >= 0 && H > 0, "stream_norm: bad sizes T=%d H=%d", T, H);
    QE_REQUIRE(H <= 15360 || (H % 4 == 0 && H <= 8192), "stream_norm: rows of %d numbers (at most 15360)", H);
    QE_REQUIRE(!delta || n_delta >= 1, "stream_norm: %d parts", n_delta);
    QE_REQUIRE(!kept || k >= 0, "stream_norm: result %d", k);
    QE_REQUIRE(!coef || kept, "stream_norm: an average over nothing");
    QE_REQUIRE(!out || w, "stream_norm: a norm without a weight");
    QE_REQUIRE(!conv_w || (out && !rows && taps >= 1 && tok_seq && (taps == 1 || state)), "stream_norm: a convolution of %d taps lacks operands", taps);
    QE_REQUIRE(rows || n_rows == T, "stream_norm: %d of %d rows", n_rows, T);
    QE_REQUIRE(!rows || !stats, "stream_norm: statistics go with all rows");
    if (n_rows == 0) return 0;
    const long stride = (long)T * H;
    StreamNorm a{x, delta, n_delta, stride, scale, kept, stride, k, coef, rows, w, out, stats, H, eps, center,
                 conv_w, state, tok_seq, conv_w ? taps : 1};
    if (dt_a == QE_F32 && (!delta || dt_d == QE_F32)) launch_stream_norm<float, float>(a, n_rows, stream);
    else if (dt_a == QE_BF16 && (!delta || dt_d == QE_F32)) launch_stream_norm<bf16_t, float>(a, n_rows, stream);
    else if (dt_a == QE_BF16 && dt_d == QE_BF16) launch_stream_norm<bf16_t, bf16_t>(a, n_rows, stream);
    else QE_REQUIRE(false, "stream_norm: no kernel for output type %d with part type %d", dt_a, dt_d);
    QE_LAUNCH_CHECK();
    return 0;
}

// ---- the convolution of many rows, h formed from the stream and the rows' statistics ----------------------------
#define NC_ROWS 8

// A thread: V channels, NC_ROWS consecutive rows.  prev[k - 1] holds h of the row k before; where a request begins
// (or began fewer than taps - 1 rows before) the request's state stands in: state[j] is the input at place
// (tokens so far) - (taps - 1) + j.
template <typename TA, int TAPS, int V>
__global__ __launch_bounds__(256) void norm_conv_kernel(const float* __restrict__ x, const float* __restrict__ stats,
                                                        const float* __restrict__ w, const float* __restrict__ conv_w,
                                                        const float* __restrict__ state, const int* __restrict__ tok_seq,
                                                        TA* __restrict__ out, int T, int H) {
    const int c = (blockIdx.x * blockDim.x + threadIdx.x) * V;
    if (c >= H) return;
    const int t0 = blockIdx.y * NC_ROWS;
    constexpr int n1 = TAPS - 1;
    float xv[NC_ROWS][V], wn[V], u[TAPS][V];
    auto load = [&](const float* p, float (&d)[V]) {
        if constexpr (V == 4) Vec4<float>::load(p, d);
        else d[0] = *p;
    };
#pragma unroll
    for (int i = 0; i < NC_ROWS; ++i) load(x + (long)min(t0 + i, T - 1) * H + c, xv[i]);
    load(w + c, wn);
#pragma unroll
    for (int j = 0; j < TAPS; ++j) load(conv_w + (long)j * H + c, u[j]);
    float prev[n1 > 0 ? n1 : 1][V];
    int seq = tok_seq[t0];
    if (n1 > 0) {
        int before = 0;
        while (before < n1 && t0 - 1 - before >= 0 && tok_seq[t0 - 1 - before] == seq) ++before;
        const float* st = state + (long)seq * n1 * H + c;
#pragma unroll
        for (int k = 1; k <= n1; ++k) {
            if (k <= before) {
                const float m = stats[2 * (t0 - k)], rs = stats[2 * (t0 - k) + 1];
                load(x + (long)(t0 - k) * H + c, prev[k - 1]);
#pragma unroll
                for (int e = 0; e < V; ++e) prev[k - 1][e] = (prev[k - 1][e] - m) * rs * wn[e];
            } else {
                load(st + (long)(n1 - k + before) * H, prev[k - 1]);
            }
        }
    }
#pragma unroll
    for (int i = 0; i < NC_ROWS; ++i) {
        const int t = t0 + i;
        if (t >= T) break;
        const int s = tok_seq[t];
        if (n1 > 0 && s != seq) {                          // another request begins (the same for the whole block)
            const float* st = state + (long)s * n1 * H + c;
#pragma unroll
            for (int k = 1; k <= n1; ++k) load(st + (long)(n1 - k) * H, prev[k - 1]);
        }
        seq = s;
        const float m = stats[2 * t], rs = stats[2 * t + 1];
        float h[V], o[V];
#pragma unroll
        for (int e = 0; e < V; ++e) {
            o[e] = h[e] = (xv[i][e] - m) * rs * wn[e];
#pragma unroll
            for (int k = n1; k >= 1; --k) o[e] = fmaf(u[n1 - k][e], prev[k - 1][e], o[e]);   // oldest input first
            o[e] = fmaf(u[n1][e], h[e], o[e]);
#pragma unroll
            for (int k = n1; k >= 2; --k) prev[k - 1][e] = prev[k - 2][e];
            if (n1 > 0) prev[0][e] = h[e];
        }
        if constexpr (V == 4) Vec4<TA>::store(out + (long)t * H + c, o);
        else Elem<TA>::store(out + (long)t * H + c, o[0]);
    }
}

// Any number of taps: every input is formed again for every output.
template <typename TA>
__global__ void norm_conv_any_kernel(const float* __restrict__ x, const float* __restrict__ stats, const float* __restrict__ w,
                                     const float* __restrict__ conv_w, const float* __restrict__ state,
                                     const int* __restrict__ tok_seq, TA* __restrict__ out, int T, int H, int taps) {
    const int c = blockIdx.x * blockDim.x + threadIdx.x;
    if (c >= H) return;
    const int n1 = taps - 1;
    for (long t = (long)blockIdx.y * NC_ROWS; t < T && t < (long)(blockIdx.y + 1) * NC_ROWS; ++t) {
        const int s = tok_seq[t];
        int before = 0;
        while (before < n1 && t - 1 - before >= 0 && tok_seq[t - 1 - before] == s) ++before;
        const float h = (x[t * H + c] - stats[2 * t]) * stats[2 * t + 1] * w[c];
        float o = h;
        for (int k = n1; k >= 1; --k) {
            const long q = t - k;
            const float p = k <= before ? (x[q * H + c] - stats[2 * q]) * stats[2 * q + 1] * w[c]
                                        : state[((long)s * n1 + (n1 - k + before)) * H + c];
            o = fmaf(conv_w[(long)(n1 - k) * H + c], p, o);
        }
        o = fmaf(conv_w[(long)n1 * H + c], h, o);
        Elem<TA>::store(out + t * H + c, o);
    }
}

// After the convolution: a request's state takes its last taps - 1 h.  A portion shorter than that moves the old
// entries up first; its first row's thread does all of it.  A block looks at 32 rows, of which few are a request's last.
#define NC_STATE_ROWS 32
__global__ __launch_bounds__(256) void norm_conv_state_kernel(const float* __restrict__ x, const float* __restrict__ stats,
                                                              const float* __restrict__ w, float* __restrict__ state,
                                                              const int* __restrict__ tok_seq, int T, int H, int taps) {
    const int c = blockIdx.x * blockDim.x + threadIdx.x;
    const int n1 = taps - 1;
    // every lane looks at one row: few are among their request's last taps - 1 (a request's rows are consecutive)
    const int mine = blockIdx.y * NC_STATE_ROWS + (threadIdx.x & (NC_STATE_ROWS - 1));
    const bool last = mine < T && !(mine + n1 < T && tok_seq[mine + n1] == tok_seq[mine]);
    unsigned long todo = __ballot(last) & ((1UL << NC_STATE_ROWS) - 1);
    for (; todo; todo &= todo - 1) {
        const int t = blockIdx.y * NC_STATE_ROWS + __builtin_ctzl(todo);
        const int s = tok_seq[t];
        int before = 0, after = 0;
        while (before < n1 && t - 1 - before >= 0 && tok_seq[t - 1 - before] == s) ++before;
        while (after < n1 && t + 1 + after < T && tok_seq[t + 1 + after] == s) ++after;
        if (c >= H) continue;
        float* st = state + (long)s * n1 * H + c;
        if (before + after + 1 < n1) {                     // the whole portion is shorter than the state
            if (before != 0) continue;
            const int q = after + 1;
            for (int j = 0; j + q < n1; ++j) st[(long)j * H] = st[(long)(j + q) * H];
            for (int m = 0; m < q; ++m)
                st[(long)(n1 - q + m) * H] = (x[(long)(t + m) * H + c] - stats[2 * (t + m)]) * stats[2 * (t + m) + 1] * w[c];
        } else if (after < n1) {
            st[(long)(n1 - 1 - after) * H] = (x[(long)t * H + c] - stats[2 * t]) * stats[2 * t + 1] * w[c];
        }
    }
}

// stats [T][2] = (mean, rstd) of the rows of x; conv_w [taps][H]; state [slots][taps - 1][H], read and brought up to date
extern "C" int qe_norm_conv(const float* x, const float* stats, const float* w, const float* conv_w, float* state,
                            const int* tok_seq, void* out, int T, int H, int taps, int dt_a, hipStream_t stream) {
    QE_REQUIRE(T >= 0 && H > 0 && taps >= 1, "norm_conv: bad sizes T=%d H=%d taps=%d", T, H, taps);
    QE_REQUIRE(taps == 1 || state, "norm_conv: %d taps need a state", taps);
    QE_REQUIRE(T <= 65535 * NC_ROWS, "norm_conv: %d rows in a step", T);
    QE_REQUIRE(dt_a == QE_F32 || dt_a == QE_BF16, "norm_conv: unknown output type %d", dt_a);
    if (T == 0) return 0;
    const int gy = qe_cdiv(T, NC_ROWS);
    const bool four = H % 4 == 0;
    const int lanes = four ? H / 4 : H;
    const int threads = lanes >= 256 ? 256 : 64;
#define QE_NC3(TA_, TAPS_, V_) norm_conv_kernel<TA_, TAPS_, V_><<<dim3(qe_cdiv(lanes, threads), gy), threads, 0, stream>>>(x, stats, w, conv_w, state, tok_seq, (TA_*)out, T, H)
#define QE_NC2(TA_, TAPS_) do { if (four) QE_NC3(TA_, TAPS_, 4); else QE_NC3(TA_, TAPS_, 1); } while (0)
#define QE_NC(TAPS_) do { if (dt_a == QE_F32) QE_NC2(float, TAPS_); else QE_NC2(bf16_t, TAPS_); } while (0)
    if (taps == 1) QE_NC(1);
    else if (taps == 2) QE_NC(2);
    else if (taps == 3) QE_NC(3);
    else if (taps == 4) QE_NC(4);
    else if (dt_a == QE_F32)
        norm_conv_any_kernel<float><<<dim3(qe_cdiv(H, 256), gy), 256, 0, stream>>>(x, stats, w, conv_w, state, tok_seq, (float*)out, T, H, taps);
    else
        norm_conv_any_kernel<bf16_t><<<dim3(qe_cdiv(H, 256), gy), 256, 0, stream>>>(x, stats, w, conv_w, state, tok_seq, (bf16_t*)out, T, H, taps);
#undef QE_NC
#undef QE_NC2
#undef QE_NC3
    QE_LAUNCH_CHECK();
    if (taps > 1) {
        norm_conv_state_kernel<<<dim3(qe_cdiv(H, 256), qe_cdiv(T, NC_STATE_ROWS)), 256, 0, stream>>>(x, stats, w, state, tok_seq, T, H, taps);
        QE_LAUNCH_CHECK();
    }
    return 0;
}
