// Paged attention, one wave per (token, query head), everything in 32-bit.
//
// This kernel serves every kind of row alike: a decoded token, a token of a
// prompt portion, a token of a whole prompt.  A token at position p of its
// request reads the keys 0..p (or the last `window` of them) of that request
// through the block table; the keys of its own step are already in the cache,
// because the cache write precedes attention inside a layer.  Keys are walked
// in ascending order in tiles of 64 with a running maximum and sum, so the
// result for a position does not depend on how the request was cut into steps
// or on what else is in the batch.  It is the attention of the true 32-bit
// path and the fallback for shapes the matrix-core kernels refuse.
//
// Two optional extras, a number a query head each: `slopes` (slope_h * (i - j) is taken off the score of key
// j for the query at position i) and `sinks` (exp(sink_h) joins the softmax's denominator once: a score
// that is not scaled and has no key and no value).  `more` (PlAttentionMore): a soft cap on the scores, first keys
// that every later query sees beside its window, and a gate a head on the read-out.  Key and value pool may be one and the same tensor.
#include "common.hpp"

#define PL_MAX_HEAD_DIM 1024

// REGS: output elements a lane (head sizes up to 64 * REGS).
template <typename T, int REGS>
__global__ void __launch_bounds__(PL_WAVE)
paged_attention_plain_kernel(const T* __restrict__ q, int q_stride, T* __restrict__ out,
                             const int* __restrict__ positions, const int* __restrict__ seq_of,
                             const int* __restrict__ block_table, int max_blocks, int block_size,
                             const T* k_pool, const T* v_pool, int nq,
                             int nkv, int d, float scale, int window, const float* __restrict__ sinks,
                             const float* __restrict__ slopes, PlAttentionMore more) {
    __shared__ float qs[REGS * PL_WAVE];
    const int t = blockIdx.x;
    const int h = blockIdx.y;
    const int lane = threadIdx.x;
    const int pos = positions[t];
    if (pos < 0) return;  // padding row

    const int kvh = h / (nq / nkv);
    const T* qrow = q + static_cast<size_t>(t) * q_stride + static_cast<size_t>(h) * d;
    for (int i = lane; i < d; i += PL_WAVE) qs[i] = to_float(qrow[i]);
    __syncthreads();

    const int* table = block_table + static_cast<size_t>(seq_of[t]) * max_blocks;
    const int first = pl_first_visible(pos, window);
    const float slope = slopes != nullptr ? slopes[h] : 0.f;

    float m = -INFINITY, l = 0.f;
    float acc[REGS];
#pragma unroll
    for (int r = 0; r < REGS; ++r) acc[r] = 0.f;

    // first the kept keys in front of the window, then the window's
    const int kept = min(more.keep, first);
    for (int j0 = kept > 0 ? 0 : first, next; j0 <= pos; j0 = next) {
        const bool front = j0 < kept;
        const int stop = front ? kept - 1 : pos;           // the last key of this stretch
        next = front && j0 + PL_WAVE >= kept ? first : j0 + PL_WAVE;
        const int j = j0 + lane;
        float s = -INFINITY;
        int slot = -1;
        if (j <= stop) {
            const int blk = table[j / block_size];
            if (blk >= 0) {
                slot = blk * block_size + j % block_size;
                const T* krow = k_pool + (static_cast<size_t>(slot) * nkv + kvh) * d;
                float dot = 0.f;
                for (int i = 0; i < d; ++i) dot = fmaf(qs[i], to_float(krow[i]), dot);
                s = dot * scale;
                if (more.cap > 0.f) s = more.cap * tanhf(s / more.cap);
                s -= slope * static_cast<float>(pos - j);
            }
        }
        const float tile_max = wave_max(s);
        const float m_new = fmaxf(m, tile_max);
        if (m_new == -INFINITY) continue;  // nothing visible yet (the same for every lane)
        const float corr = expf(m - m_new);  // exp(-inf) = 0 on the first tile
        const float p = (slot >= 0) ? expf(s - m_new) : 0.f;
        l = l * corr + wave_sum(p);
#pragma unroll
        for (int r = 0; r < REGS; ++r) acc[r] *= corr;
        const int count = min(PL_WAVE, stop - j0 + 1);
        for (int jj = 0; jj < count; ++jj) {
            const float pj = __shfl(p, jj, PL_WAVE);
            const int sj = __shfl(slot, jj, PL_WAVE);
            if (sj < 0) continue;
            const T* vrow = v_pool + (static_cast<size_t>(sj) * nkv + kvh) * d;
#pragma unroll
            for (int r = 0; r < REGS; ++r) {
                const int i = lane + r * PL_WAVE;
                if (i < d) acc[r] = fmaf(pj, to_float(vrow[i]), acc[r]);
            }
        }
        m = m_new;
    }
    if (sinks != nullptr) {
        // one more term of the denominator, with no value behind it
        const float sink = sinks[h];
        const float m_new = fmaxf(m, sink);
        const float corr = expf(m - m_new);
        l = l * corr + expf(sink - m_new);
#pragma unroll
        for (int r = 0; r < REGS; ++r) acc[r] *= corr;
    }
    const float opened = more.gate != nullptr ? pl_head_gate(more, t, h) : 1.f;
    T* orow = out + (static_cast<size_t>(t) * nq + h) * d;
#pragma unroll
    for (int r = 0; r < REGS; ++r) {
        const int i = lane + r * PL_WAVE;
        if (i < d) orow[i] = from_float<T>(l > 0.f ? acc[r] / l * opened : 0.f);
    }
}

extern "C" int pl_paged_attention_plain(const void* q, int q_stride, void* out, const int* positions,
                                        const int* seq_of, const int* block_table, int max_blocks,
                                        int block_size, const void* k_pool, const void* v_pool, int n,
                                        int nq, int nkv, int d, float scale, int window, int dtype,
                                        const float* sinks, const float* slopes, float cap, int keep,
                                        const float* gate, int gate_stride, hipStream_t stream) {
    PL_REQUIRE(cap >= 0.f && keep >= 0 && (gate == nullptr || gate_stride >= nq), "attention: a cap of %g, %d first keys kept, gates in rows of %d",
               static_cast<double>(cap), keep, gate_stride);
    PL_REQUIRE(keep == 0 || window >= 0, "attention: first keys kept beside blocks of positions");
    const PlAttentionMore more{cap, keep, gate, gate_stride};
    PL_REQUIRE(d > 0 && d <= PL_MAX_HEAD_DIM, "attention: head size %d, which has to be between 1 and %d", d, PL_MAX_HEAD_DIM);
    PL_REQUIRE(nq > 0 && nkv > 0 && nq % nkv == 0, "attention: %d query heads over %d key heads", nq, nkv);
    PL_REQUIRE(block_size > 0 && max_blocks > 0 && q_stride >= nq * d,
               "attention: block size %d, %d blocks a row, query stride %d, window %d", block_size, max_blocks, q_stride, window);
    PL_REQUIRE(nq <= 65535, "attention: %d query heads are more than one launch covers", nq);
    if (n <= 0) return 0;
    dim3 grid(n, nq);
#define PL_PLAIN_LAUNCH(T, REGS)                                                                                        \
    paged_attention_plain_kernel<T, REGS><<<grid, PL_WAVE, 0, stream>>>(                                                \
        static_cast<const T*>(q), q_stride, static_cast<T*>(out), positions, seq_of, block_table, max_blocks,          \
        block_size, static_cast<const T*>(k_pool), static_cast<const T*>(v_pool), nq, nkv, d, scale, window, sinks,    \
        slopes, more)
    if (dtype == PL_DTYPE_F32) {
        if (d <= 256) PL_PLAIN_LAUNCH(float, 4);
        else PL_PLAIN_LAUNCH(float, 16);
    } else if (dtype == PL_DTYPE_BF16) {
        if (d <= 256) PL_PLAIN_LAUNCH(bf16_t, 4);
        else PL_PLAIN_LAUNCH(bf16_t, 16);
    } else {
        PL_REQUIRE(false, "attention: dtype code %d", dtype);
    }
#undef PL_PLAIN_LAUNCH
    PL_CHECK_LAUNCH("paged_attention_plain");
    return 0;
}
