// Attention of a flat batch of new tokens over the paged cache, any sizes, all
// arithmetic in 32-bit.  One wave per (token, query head).  (The fallback of the bfloat16 mode for
// sizes the MFMA kernels refuse, and of the float32 mode for head sizes that are no multiple of 16;
// float32 otherwise goes to attention_f32.hip.)
//
// The query of token t at absolute position p = positions[t] of request
// s = tok_seq[t] sees the keys at positions lo..p of that request, read through
// block_table[s]; lo = 0, or p - window + 1 when a window is given.  With keep_first the
// request's first keep_first keys are seen as well, wherever the window stands.  Keys are
// taken 64 at a time, the kept first keys behind the window first, then from lo upwards, with
// an online softmax, so the order of the sums depends on p, the window and keep_first only:
// not on how the request's tokens were cut into steps, nor on what else is in the batch.
// With sink the softmax has one more entry that carries no value, of the head's score in AttnTail or of score 0:
// the running maximum starts there with a sum of 1.
//
// cache of one layer: [page][2 (k, v)][Hkv][P * D]; a key tile is [P][D], a value tile is
// stored transposed, [D][P] (the layout the MFMA kernels read without a shuffle).
#include "common.h"

#define ATTN_MAX_D 256

template <typename TA>
__global__ __launch_bounds__(64) void attention_generic_kernel(
    const TA* __restrict__ q, TA* __restrict__ out, const TA* __restrict__ cache,
    const int* __restrict__ positions, const int* __restrict__ tok_seq,
    const int* __restrict__ block_table, int max_blocks, const int* __restrict__ tokens,
    int Hq, int Hkv, int D, int P, float scale, int window, int keep_first, int sink, float softcap, AttnTail tail) {
    extern __shared__ float smem[];
    float* qs = smem;            // D
    float* ps = smem + D;        // 64 probabilities of the current chunk
    long* voff = (long*)(smem + ((D + 64 + 1) & ~1));  // 64 offsets of the chunk's value rows
    const long t = tokens ? tokens[blockIdx.x] : blockIdx.x;   // a subset of the batch, or all of it
    const int h = blockIdx.y;
    const int lane = threadIdx.x;
    const int kvh = h / (Hq / Hkv);
    const int p_own = positions[t];
    const int* bt = block_table + (long)tok_seq[t] * max_blocks;
    const int lo = first_seen_key(p_own, window);
    const long page_stride = 2L * Hkv * P * D;

    const TA* qrow = q + (t * Hq + h) * D;
    for (int d = lane; d < D; d += 64) qs[d] = Elem<TA>::load(qrow + d);
    __syncthreads();

    float m = sink ? tail.sink_of(h) : -INFINITY, l = sink ? 1.f : 0.f;
    float acc[ATTN_MAX_D / 64];
#pragma unroll
    for (int i = 0; i < ATTN_MAX_D / 64; ++i) acc[i] = 0.f;

    // two walks: the kept first keys that lie behind the window, 0 .. kf - 1, then lo .. p
    const int kf = keep_first < lo ? keep_first : lo;
    for (int walk = kf > 0 ? 0 : 1; walk < 2; ++walk)
    for (int j0 = walk ? lo : 0, p = walk ? p_own : kf - 1; j0 <= p; j0 += 64) {
        const int j = j0 + lane;
        float sc = -INFINITY;
        long vo = 0;
        if (j <= p) {
            const long page = bt[j / P];
            const int off = j % P;
            const long kbase = page * page_stride + ((long)kvh * P + off) * D;
            vo = page * page_stride + ((long)(Hkv + kvh) * P) * D + off;   // + d * P
            const TA* krow = cache + kbase;
            float dot = 0.f;
            for (int d = 0; d < D; ++d) dot = fmaf(qs[d], Elem<TA>::load(krow + d), dot);
            sc = dot * scale;
            if (softcap > 0.f) sc = softcap * tanhf(sc / softcap);
        }
        const float mn = fmaxf(m, wave_max(sc));   // finite: key j0 is always seen
        const float alpha = expf(m - mn);          // exp(-inf) = 0 on the first chunk
        const float pj = (j <= p) ? expf(sc - mn) : 0.f;
        l = l * alpha + wave_sum(pj);
        m = mn;
        ps[lane] = pj;
        voff[lane] = vo;
        __syncthreads();
        const int cnt = (p - j0 + 1 < 64) ? p - j0 + 1 : 64;
#pragma unroll
        for (int i = 0; i < ATTN_MAX_D / 64; ++i) {
            const int d = lane + i * 64;
            if (d < D) {
                float a = acc[i] * alpha;
                for (int jj = 0; jj < cnt; ++jj)
                    a = fmaf(ps[jj], Elem<TA>::load(cache + voff[jj] + (long)d * P), a);
                acc[i] = a;
            }
        }
        __syncthreads();
    }
    const float inv = 1.f / l;
#pragma unroll
    for (int i = 0; i < ATTN_MAX_D / 64; ++i) {
        const int d = lane + i * 64;
        if (d < D) tail.store(out, t, h, d, acc[i] * inv);
    }
}

bool qe_attention_f32_ok(int Hq, int Hkv, int D, int P);
int qe_attention_f32(const float* q, float* out, const float* cache, const int* positions, const int* tok_seq,
                     const int* block_table, int max_blocks, const int* tokens, int T, int Hq, int Hkv, int D,
                     int P, float scale, int window, int keep_first, int sink, float softcap, hipStream_t stream, const AttnTail& tail);

// 32-bit attention goes to the kernel on the matrix units (attention_f32.hip) where it takes the
// sizes, unless qe_use_matrix_f32(0) has switched that off.
extern int g_qe_matrix_f32;

int qe_attention_generic(const void* q, void* out, const void* cache, const int* positions,
                         const int* tok_seq, const int* block_table, int max_blocks, const int* tokens,
                         int T, int Hq, int Hkv, int D, int P, float scale, int window, int keep_first, int sink,
                         float softcap, int dt_a, hipStream_t stream, const AttnTail& tail) {
    if (dt_a == QE_F32 && g_qe_matrix_f32 && qe_attention_f32_ok(Hq, Hkv, D, P))
        return qe_attention_f32((const float*)q, (float*)out, (const float*)cache, positions, tok_seq, block_table,
                                max_blocks, tokens, T, Hq, Hkv, D, P, scale, window, keep_first, sink, softcap, stream, tail);
    QE_REQUIRE(D <= ATTN_MAX_D, "attention: head_dim=%d exceeds %d", D, ATTN_MAX_D);
    QE_REQUIRE(Hq <= 65535, "attention: too many heads");
    dim3 grid(T, Hq);
    const size_t shmem = (size_t)((D + 64 + 1) & ~1) * sizeof(float) + 64 * sizeof(long);
    if (dt_a == QE_F32)
        attention_generic_kernel<float><<<grid, 64, shmem, stream>>>(
            (const float*)q, (float*)out, (const float*)cache, positions, tok_seq, block_table,
            max_blocks, tokens, Hq, Hkv, D, P, scale, window, keep_first, sink, softcap, tail);
    else if (dt_a == QE_BF16)
        attention_generic_kernel<bf16_t><<<grid, 64, shmem, stream>>>(
            (const bf16_t*)q, (bf16_t*)out, (const bf16_t*)cache, positions, tok_seq, block_table,
            max_blocks, tokens, Hq, Hkv, D, P, scale, window, keep_first, sink, softcap, tail);
    else
        QE_REQUIRE(false, "attention: unknown dtype %d", dt_a);
    QE_LAUNCH_CHECK();
    return 0;
}
