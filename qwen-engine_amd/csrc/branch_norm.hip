// What stands between one sublayer and the next where a layer norms what its sublayers give as well as what they read:
//
//   y = scale * (a_0 + a_1 + ...)                              the branch's parts
//   x <- x + mult * y * rsqrt(mean(y^2) + eps_y) * w_y         the residual sum on the 32-bit stream
//   out = x * rsqrt(mean(x^2) + eps) * w                       the norm before the next sublayer (if asked for)
//
// in one pass over the row.  Parts are added in ascending order; everything is 32-bit with one rounding at the store.
// With rows only those rows are formed and nothing is written back (the model's last norm on the wanted rows).
#include "common.h"

struct BranchNorm {
    float* x;                      // [T, H]
    const void* a;                 // n_a tensors [T, H], one after the other
    int n_a;
    float sa;
    long stride;                   // T * H
    const float* w_y;
    float eps_y, mult;
    const int* rows;
    const float* w;                // or null: no norm behind the sum
    float eps;
    void* out;
    int H;
};

template <typename TD>
__device__ __forceinline__ float branch_at(const BranchNorm& p, long at) {
    float y = 0.f;
    for (int s = 0; s < p.n_a; ++s) y += Elem<TD>::load((const TD*)p.a + s * p.stride + at);
    y *= p.sa;
    return y;
}

// Any row length: three passes, the branch formed again in each.
template <typename TA, typename TD>
__global__ __launch_bounds__(256) void branch_norm_kernel(BranchNorm p) {
    __shared__ float red[16];
    const long r = blockIdx.x, src = p.rows ? (long)p.rows[r] : r;
    const int H = p.H;
    float* xr = p.x + src * H;
    float ss = 0.f;
    for (int c = threadIdx.x; c < H; c += blockDim.x) {
        const float y = branch_at<TD>(p, src * H + c);
        ss += y * y;
    }
    const float fy = p.mult * rsqrtf(block_sum(ss, red) / (float)H + p.eps_y);
    ss = 0.f;
    for (int c = threadIdx.x; c < H; c += blockDim.x) {
        const float v = fmaf(branch_at<TD>(p, src * H + c) * fy, p.w_y[c], xr[c]);
        ss += v * v;
    }
    ss = block_sum(ss, red);                               // (and the rows' last readers of x are done)
    const float f = rsqrtf(ss / (float)H + p.eps);
    for (int c = threadIdx.x; c < H; c += blockDim.x) {
        const float v = fmaf(branch_at<TD>(p, src * H + c) * fy, p.w_y[c], xr[c]);
        if (!p.rows) xr[c] = v;
        if (p.w) Elem<TA>::store((TA*)p.out + r * H + c, v * f * p.w[c]);
    }
}

// H a multiple of 4, up to NV * 4 * blockDim.x numbers: the row stays in registers.  FEW: few rows, whose time is the
// latency of their loads: SB parts at a time, the stream and both weights are asked for before anything is waited for,
// from addresses that are always valid (a piece beyond the row or a part beyond the last reads another again and is not
// used).  Many rows are bound by the memory's rate.
template <typename TA, typename TD, int NV, bool FEW>
__global__ __launch_bounds__(256) void branch_norm_regs_kernel(BranchNorm p) {
    constexpr int SB = !FEW ? 2 : (NV <= 2 ? 8 : 4);
    __shared__ float red[2][16];
    const long r = blockIdx.x, src = p.rows ? (long)p.rows[r] : r;
    const int H = p.H;
    float* xr = p.x + src * H;
    int cs[NV];
    bool ok[NV];
#pragma unroll
    for (int i = 0; i < NV; ++i) {
        const int c = (threadIdx.x + i * blockDim.x) * 4;
        ok[i] = c < H;
        cs[i] = ok[i] ? c : 0;
    }
    float y[NV][4], x[NV][4], wy[NV][4], w[NV][4];
#pragma unroll
    for (int i = 0; i < NV; ++i) {
        Vec4<float>::load(xr + cs[i], x[i]);
        Vec4<float>::load(p.w_y + cs[i], wy[i]);
        if (p.w) Vec4<float>::load(p.w + cs[i], w[i]);
#pragma unroll
        for (int e = 0; e < 4; ++e) y[i][e] = 0.f;
    }
    for (int s0 = 0; s0 < p.n_a; s0 += SB) {
        float d[SB][NV][4];
#pragma unroll
        for (int s = 0; s < SB; ++s) {
            if (!FEW && s0 + s >= p.n_a) continue;
            const TD* part = (const TD*)p.a + (long)min(s0 + s, p.n_a - 1) * p.stride + src * H;
#pragma unroll
            for (int i = 0; i < NV; ++i) Vec4<TD>::load(part + cs[i], d[s][i]);
        }
#pragma unroll
        for (int s = 0; s < SB; ++s)
            if (s0 + s < p.n_a) {
#pragma unroll
                for (int i = 0; i < NV; ++i)
#pragma unroll
                    for (int e = 0; e < 4; ++e) y[i][e] += d[s][i][e];
            }
    }
#pragma unroll
    for (int i = 0; i < NV; ++i)
#pragma unroll
        for (int e = 0; e < 4; ++e) y[i][e] *= p.sa;
    float ss = 0.f;
#pragma unroll
    for (int i = 0; i < NV; ++i)
        if (ok[i]) {
#pragma unroll
            for (int e = 0; e < 4; ++e) ss += y[i][e] * y[i][e];
        }
    const float fy = p.mult * rsqrtf(block_sum(ss, red[0]) / (float)H + p.eps_y);
    ss = 0.f;
#pragma unroll
    for (int i = 0; i < NV; ++i)
        if (ok[i]) {
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                x[i][e] = fmaf(y[i][e] * fy, wy[i][e], x[i][e]);
                ss += x[i][e] * x[i][e];
            }
            if (!p.rows) Vec4<float>::store(xr + cs[i], x[i]);
        }
    if (!p.w) return;
    const float f = rsqrtf(block_sum(ss, red[1]) / (float)H + p.eps);
#pragma unroll
    for (int i = 0; i < NV; ++i)
        if (ok[i]) {
            float o[4];
#pragma unroll
            for (int e = 0; e < 4; ++e) o[e] = x[i][e] * f * w[i][e];
            Vec4<TA>::store((TA*)p.out + r * H + cs[i], o);
        }
}

// n_rows: rows to form (T, or the length of rows).  dt_d: element type of a; dt_a: of out.
extern "C" int qe_branch_norm(float* x, const void* a, int n_a, float scale, int dt_d,
                              const float* w_y, float eps_y, float mult, const int* rows, int n_rows, const float* w, float eps,
                              void* out, int dt_a, int T, int H, hipStream_t stream) {
    QE_REQUIRE(T >= 0 && H > 0 && n_rows >= 0, "branch_norm: bad sizes T=%d H=%d", T, H);
    QE_REQUIRE(a && n_a >= 1 && w_y && (!w || out), "branch_norm: no branch, or no place for the normed rows");
    if (n_rows == 0) return 0;
    BranchNorm p{x, a, n_a, scale, (long)T * H, w_y, eps_y, mult, rows, w, eps, out, H};
    const bool regs = H % 4 == 0 && H <= 8192;
    const int threads = regs ? (qe_cdiv(H / 4, 64) * 64 > 256 ? 256 : qe_cdiv(H / 4, 64) * 64) : 256;
    const int nv = regs ? qe_cdiv(H / 4, threads) : 0;
    const bool few = n_rows <= 512;
#define QE_BN3(TA_, TD_, NV_) do { if (few) branch_norm_regs_kernel<TA_, TD_, NV_, true><<<n_rows, threads, 0, stream>>>(p); \
                                   else branch_norm_regs_kernel<TA_, TD_, NV_, false><<<n_rows, threads, 0, stream>>>(p); } while (0)
#define QE_BN(TA_, TD_)                                                                        \
    do {                                                                                       \
        if (!regs) branch_norm_kernel<TA_, TD_><<<n_rows, threads, 0, stream>>>(p);            \
        else if (nv <= 1) QE_BN3(TA_, TD_, 1);                                                 \
        else if (nv <= 2) QE_BN3(TA_, TD_, 2);                                                 \
        else if (nv <= 4) QE_BN3(TA_, TD_, 4);                                                 \
        else QE_BN3(TA_, TD_, 8);                                                              \
    } while (0)
    if (dt_a == QE_F32 && dt_d == QE_F32) QE_BN(float, float);
    else if (dt_a == QE_BF16 && dt_d == QE_F32) QE_BN(bf16_t, float);
    else if (dt_a == QE_BF16 && dt_d == QE_BF16) QE_BN(bf16_t, bf16_t);
    else if (dt_a == QE_F32 && dt_d == QE_BF16) QE_BN(float, bf16_t);
    else QE_REQUIRE(false, "branch_norm: no kernel for branches of type %d and rows of type %d", dt_d, dt_a);
#undef QE_BN
#undef QE_BN3
    QE_LAUNCH_CHECK();
    return 0;
}
