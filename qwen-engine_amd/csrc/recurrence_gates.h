// Activations and gates that the kernels of the recurrences apply as they read their operands, all in 32-bit.
#pragma once
#include "common.h"

// The operands of the recurrences' kernels (the binding mirrors this layout).  Row t of q and k: Hk heads of D numbers,
// head h of the H value heads using q/k head h / (H / Hk); of v: H heads of Dv.
//   mode 0: decay [H]                     S <- decay_h S + k v^T                                o = S^T q
//   mode 1: wx [T][H * D] before the exponentials, w0 and u [H * D]     o = (S + diag(u) k v^T)^T q, then S <- diag(w) S + k v^T
//   mode 2: k holds a forget gate's logits, w0 its bias, u its lower bound [H * D]   S <- diag(f) S + (1 - f) v^T   o = S^T q
//   mode 3: wx [T][H * D] the decays themselves                         S <- diag(w) S + k v^T  o = S^T q
//   mode 4: wx [T][H] one decay a row and head, ks [T][H] a factor on the key     S <- w S + (ks k) v^T  o = S^T q
//           (number (t, h) of wx, ks and fl at t * w_stride + h * w_head)
//   mode 5: as 4, and n <- w n + ks k; o = S^T q / (max(|n . q|, fl) + 1e-6) with fl [T][H]
// q is multiplied by q_scale.  act_silu: q, k and v (mode 2: q) pass silu as they are read.
// A request's state: H * D * Dv numbers; in mode 5 then rec_copies(Dv) equal copies of n [H][D] (a block of value columns
// reads and writes its own).
// Where every row is the only row of its request the kernel forms the decays of modes 3 and 5 itself from what they come
// from: mode 3 from low (dt_low, rank numbers a row), w2 [rank][H * D], b2 and inv_tau (low_rank_decay below); mode 5 from the
// gates' logits z [T][2 H], ib, fb, cap and the running maxima at state + m_at + h (memory_gates_of below).
// Results: out float32 [T][H][Dv]; or, with norm_w [H * Dv], every head's o divided by its root mean square (norm_eps
// inside), times the weight, times act(gate) (gate_act 1 silu, 2 sigmoid; number h * Dv + c of the gate's row), times
// y_scale, in dt_y at y + t * y_stride + h * Dv.
struct Rec {
    const void* q;
    const void* k;
    const void* v;
    long row_stride;
    const float* wx;
    const float* ks;
    const float* fl;
    long w_stride;                  // of wx, ks and fl: from row to row
    long w_head;                    // and (modes 4 and 5) from head to head
    const float* w0;
    const float* u;
    const float* decay;
    float* state;
    long state_stride;
    const int* tok_seq;
    float* out;
    const float* norm_w;
    void* y;
    long y_stride;
    const void* gate;
    long gate_stride;
    const int* chunks;
    const int* portions;
    float* ws;
    const void* low;
    long low_stride;
    const float* w2;
    const float* b2;
    const float* z;
    long z_stride;
    const float* ib;
    const float* fb;
    long m_at;
    float norm_eps, q_scale, y_scale, inv_tau, cap;
    int rank, dt_low;
    int mode, act_silu, dt_a, dt_y, dt_g, gate_act, T, H, Hk, D, Dv, n_chunks, n_portions, all_single;
};

__host__ __device__ __forceinline__ int rec_copies(int Dv) { return (Dv + 63) / 64; }
__host__ __device__ __forceinline__ long rec_state_numbers(int mode, int H, int D, int Dv) {
    return (long)H * D * Dv + (mode == 5 ? (long)rec_copies(Dv) * H * D : 0);
}
static inline bool rec_operands_ok(const Rec& a, bool single) {
    switch (a.mode) {
        case 0: return a.decay != nullptr;
        case 1: return a.wx && a.w0 && a.u;
        case 2: return a.w0 && a.u;
        case 3: return a.wx || (single && a.low && a.w2 && a.b2 && a.rank > 0);
        case 4: return a.wx && a.ks;
        case 5: return (a.wx && a.ks && a.fl) || (single && a.z && a.ib && a.fb && a.cap > 0.f);
    }
    return false;
}
#define QE_REC_CHECK(a, what, single)                                                                                            \
    QE_REQUIRE((a).T >= 0 && (a).H > 0 && (a).H <= 65535 && (a).D > 0 && (a).D <= 256 && (a).Dv > 0, what ": bad sizes (heads of %d x %d)", (a).D, (a).Dv); \
    QE_REQUIRE((a).Hk > 0 && (a).H % (a).Hk == 0 && ((a).mode == 4 || (a).Hk == (a).H), what ": %d heads over %d", (a).H, (a).Hk); \
    QE_REQUIRE(rec_operands_ok(a, single), what ": mode %d lacks operands", (a).mode);                                              \
    QE_REQUIRE((a).state && (a).state_stride >= rec_state_numbers((a).mode, (a).H, (a).D, (a).Dv), what ": state rows overlap"); \
    QE_REQUIRE((a).dt_a == QE_F32 || (a).dt_a == QE_BF16, what ": unknown element type %d", (a).dt_a);                      \
    QE_REQUIRE(!(a).norm_w || ((a).y && (a).y_stride >= (long)(a).H * (a).Dv && ((a).dt_y == QE_F32 || (a).dt_y == QE_BF16)), what ": no place for the normed rows"); \
    QE_REQUIRE(!(a).gate || ((a).norm_w && (a).gate_stride >= (long)(a).H * (a).Dv && ((a).dt_g == QE_F32 || (a).dt_g == QE_BF16)), what ": a gate goes with the norm")

__device__ __forceinline__ float silu_f(float z) { return z / (1.f + expf(-z)); }
__device__ __forceinline__ float sigmoid_f(float z) { return 1.f / (1.f + expf(-z)); }
// sigmoid(z) and sigmoid(-z), neither by a difference.  exp(-|z|) from the hardware's exponential of base 2 with the
// rounding of the argument's product put back (a few parts in 10^7; nothing here overflows: the argument is not positive).
__device__ __forceinline__ void sigmoid_both(float z, float& pos, float& neg) {
    const float x = -fabsf(z);
    const float t = x * 1.44269502f;                         // log2(e), high part
    const float lost = fmaf(x, 1.92596303e-8f, fmaf(x, 1.44269502f, -t));
    const float e0 = __builtin_amdgcn_exp2f(t);
    const float e = fmaf(e0 * 0.693147182f, lost, e0);
    const float big = __builtin_amdgcn_rcpf(1.f + e), small = e * big;
    pos = z >= 0.f ? big : small;
    neg = z >= 0.f ? small : big;
}
__device__ __forceinline__ float silu_quick(float z) {
    float p, n;
    sigmoid_both(z, p, n);
    return z * p;
}
// f = l + (1 - l) sigmoid(z) and 1 - f
__device__ __forceinline__ void forget_gate(float z, float l, float& f, float& kf) {
    float p, n;
    sigmoid_both(z, p, n);
    f = fmaf(1.f - l, p, l);
    kf = (1.f - l) * n;
}

__device__ __forceinline__ float log_sigmoid(float z) { return fminf(z, 0.f) - log1pf(expf(-fabsf(z))); }
// The log gates of a matrix memory from their logits (the biases added): i = cap * tanh(zi / cap), f = log sigmoid(cap *
// tanh(zf / cap)).
__device__ __forceinline__ void memory_gates_of(float zi, float zf, float cap, float& i, float& f) {
    i = cap * tanhf(zi / cap);
    f = log_sigmoid(cap * tanhf(zf / cap));
}
// sigmoid(z)^(1 / tau), from the hardware's exponential and logarithm of base 2: the argument of the last exponential is good
// to some 1e-7 of 1 + |z|, and so is the decay
__device__ __forceinline__ float low_rank_decay(float z, float inv_tau) {
    const float l2e = 1.44269504f;
    const float t = __builtin_amdgcn_exp2f(-fabsf(z) * l2e);
    return __builtin_amdgcn_exp2f((fminf(z, 0.f) * l2e - __builtin_amdgcn_logf(1.f + t)) * inv_tau);
}

// what the gate of an output is: act(z), act 1 silu, 2 sigmoid
__device__ __forceinline__ float gate_value(float z, int act) {
    const float p = 1.f / (1.f + expf(-z));
    return act == 1 ? z * p : p;
}
__device__ __forceinline__ float rec_gate(const Rec& a, long row, int at) {
    const long i = row * a.gate_stride + at;
    return a.dt_g == QE_F32 ? ((const float*)a.gate)[i] : bf16_to_float(((const bf16_t*)a.gate)[i]);
}
__device__ __forceinline__ void rec_store(const Rec& a, long row, int at, float v) {
    const long i = row * a.y_stride + at;
    if (a.dt_y == QE_BF16) ((bf16_t*)a.y)[i] = float_to_bf16(v);
    else ((float*)a.y)[i] = v;
}
