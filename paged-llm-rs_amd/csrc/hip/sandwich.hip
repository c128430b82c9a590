// Layers whose sublayers stand between two norms, and an embedding that looks at the token before.
//
// sandwich_step: one pass over a row of the 32-bit stream, either half optional.  First what a sublayer gave
// joins the stream through the norm behind it, x <- x + norm(y); then the norm in front of the next sublayer
// reads the updated row, out = norm(x), rounded once into the model's type.  A norm is a layer norm
// ((x - mean) / sqrt(mean((x - mean)^2) + eps)) or an RMS norm (x / sqrt(mean(x^2) + eps)), times a gain a column,
// plus, where there is one, a bias a column.  Statistics, gains, biases and sums are 32-bit; the variance is the
// mean of the squared deviations, taken in a pass of its own over the registers that hold the row.
//
// bigram_add: a row of a second table joins the stream, chosen by a token and the one before it.
#include "common.hpp"

struct SandwichArgs {
    float* resid;            // [n, W]
    const float* y;          // [n, W] or null: nothing joins the stream
    const float* gain_y;     // [W]: the norm of y
    const float* bias_y;     // [W] or null
    float eps_y;
    const float* gain_x;     // [W] or null: no rows are normed
    const float* bias_x;
    float eps_x;
    void* out;               // [rows, W]
    const int* rows;         // the rows to norm (then nothing joins), or null for all
    int W;
};

// Sum over the workgroup; every thread gets it.  `scratch`: sixteen floats of LDS that no other sum of the kernel uses.
__device__ __forceinline__ float sandwich_sum(float v, float* scratch) {
    const int lane = threadIdx.x % PL_WAVE, wave = threadIdx.x / PL_WAVE, waves = blockDim.x / PL_WAVE;
    v = wave_sum(v);
    if (waves == 1) return v;
    if (lane == 0) scratch[wave] = v;
    __syncthreads();
    float total = 0.f;
    for (int w = 0; w < waves; ++w) total += scratch[w];
    return total;
}

// A workgroup a row; a thread holds RUNS runs of PER neighbouring columns in registers from the first load to the last store.
template <typename T, int PER, int RUNS, bool CENTRED>
__global__ __launch_bounds__(1024) void sandwich_step_kernel(SandwichArgs a) {
    __shared__ float scratch[4][16];
    typedef float vec_t __attribute__((ext_vector_type(PER)));
    const int i = blockIdx.x, W = a.W;
    const size_t in_row = static_cast<size_t>(a.rows != nullptr ? a.rows[i] : i) * W;
    float* x = a.resid + in_row;
    const bool joins = a.y != nullptr, reads = a.gain_x != nullptr;
    vec_t xv[RUNS], yv[RUNS], gy[RUNS], by[RUNS], gx[RUNS], bx[RUNS];
    bool in[RUNS];
#pragma unroll
    for (int k = 0; k < RUNS; ++k) {
        const int c = (threadIdx.x + k * blockDim.x) * PER;
        in[k] = c < W;
        const int cc = in[k] ? c : 0;
        xv[k] = *reinterpret_cast<const vec_t*>(x + cc);
        yv[k] = gy[k] = by[k] = gx[k] = bx[k] = vec_t(0.f);
        if (joins) {
            yv[k] = *reinterpret_cast<const vec_t*>(a.y + in_row + cc);
            gy[k] = *reinterpret_cast<const vec_t*>(a.gain_y + cc);
            if (a.bias_y != nullptr) by[k] = *reinterpret_cast<const vec_t*>(a.bias_y + cc);
        }
        if (reads) {
            gx[k] = *reinterpret_cast<const vec_t*>(a.gain_x + cc);
            if (a.bias_x != nullptr) bx[k] = *reinterpret_cast<const vec_t*>(a.bias_x + cc);
        }
    }
    const float width = static_cast<float>(W);
    // (mean, 1 / sqrt(...)) of the row that v holds
    auto statistics = [&](const vec_t (&v)[RUNS], float eps, float* first, float* second, float& mean, float& inv) {
        mean = 0.f;
        if (CENTRED) {
            float sum = 0.f;
#pragma unroll
            for (int k = 0; k < RUNS; ++k)
                if (in[k]) {
#pragma unroll
                    for (int e = 0; e < PER; ++e) sum += v[k][e];
                }
            mean = sandwich_sum(sum, first) / width;
        }
        float ss = 0.f;
#pragma unroll
        for (int k = 0; k < RUNS; ++k)
            if (in[k]) {
#pragma unroll
                for (int e = 0; e < PER; ++e) ss += (v[k][e] - mean) * (v[k][e] - mean);
            }
        inv = 1.f / sqrtf(sandwich_sum(ss, second) / width + eps);
    };
    float mean, inv;
    if (joins) {
        statistics(yv, a.eps_y, scratch[0], scratch[1], mean, inv);
#pragma unroll
        for (int k = 0; k < RUNS; ++k)
            if (in[k]) {
#pragma unroll
                for (int e = 0; e < PER; ++e) xv[k][e] += (yv[k][e] - mean) * inv * gy[k][e] + by[k][e];
                *reinterpret_cast<vec_t*>(x + (threadIdx.x + k * blockDim.x) * PER) = xv[k];
            }
    }
    if (!reads) return;
    statistics(xv, a.eps_x, scratch[2], scratch[3], mean, inv);
    T* out = static_cast<T*>(a.out) + static_cast<size_t>(i) * W;
#pragma unroll
    for (int k = 0; k < RUNS; ++k)
        if (in[k]) {
            struct __attribute__((aligned(PER * sizeof(T)))) run_t { T v[PER]; };
            run_t r;
#pragma unroll
            for (int e = 0; e < PER; ++e) r.v[e] = from_float<T>((xv[k][e] - mean) * inv * gx[k][e] + bx[k][e]);
            *reinterpret_cast<run_t*>(out + (threadIdx.x + k * blockDim.x) * PER) = r;
        }
}

template <typename T, bool CENTRED>
static int launch_sandwich(const SandwichArgs& a, int n, hipStream_t stream) {
    const int W = a.W;
    if (W % 4 == 0) {
        const int quads = W / 4;
        const int runs = quads <= 1024 ? 1 : (quads <= 2048 ? 2 : 4);
        const int threads = (pl_ceil_div(quads, runs) + 63) / 64 * 64;
        if (runs == 1) sandwich_step_kernel<T, 4, 1, CENTRED><<<n, threads, 0, stream>>>(a);
        else if (runs == 2) sandwich_step_kernel<T, 4, 2, CENTRED><<<n, threads, 0, stream>>>(a);
        else sandwich_step_kernel<T, 4, 4, CENTRED><<<n, threads, 0, stream>>>(a);
    } else {
        const int runs = W <= 4096 ? 4 : 16;
        const int threads = (pl_ceil_div(W, runs) + 63) / 64 * 64;
        if (runs == 4) sandwich_step_kernel<T, 1, 4, CENTRED><<<n, threads, 0, stream>>>(a);
        else sandwich_step_kernel<T, 1, 16, CENTRED><<<n, threads, 0, stream>>>(a);
    }
    PL_CHECK_LAUNCH("sandwich_step");
    return 0;
}

// resid [*, W] (32-bit) in place; y [n, W] (32-bit) with its norm's gain, bias (or null) and eps, or null; gain_x, bias_x
// (or null), eps_x: the norm of the updated rows, into out [n, W] in `dtype`, or gain_x null for none.  centred: 1 layer
// norms, 0 RMS norms.  rows: the n rows to norm (nothing joins the stream then).
extern "C" int pl_sandwich_step(float* resid, const float* y, const float* gain_y, const float* bias_y, float eps_y,
                                const float* gain_x, const float* bias_x, float eps_x, void* out, int dtype,
                                const int* rows, int centred, int n, int W, hipStream_t stream) {
    PL_REQUIRE(n >= 0 && W > 0 && W <= 16384, "sandwich_step: %d rows of %d (up to 16384)", n, W);
    PL_REQUIRE((y == nullptr) == (gain_y == nullptr) && (gain_x == nullptr) == (out == nullptr),
               "sandwich_step: a norm needs its rows, its gain and room for what it gives");
    PL_REQUIRE(rows == nullptr || y == nullptr, "sandwich_step: a list of rows and a sum into the stream");
    PL_REQUIRE(dtype == PL_DTYPE_F32 || dtype == PL_DTYPE_BF16, "sandwich_step: dtype code %d", dtype);
    if (n == 0 || (y == nullptr && gain_x == nullptr)) return 0;
    const SandwichArgs a{resid, y, gain_y, bias_y, eps_y, gain_x, bias_x, eps_x, out, rows, W};
    if (dtype == PL_DTYPE_F32)
        return centred ? launch_sandwich<float, true>(a, n, stream) : launch_sandwich<float, false>(a, n, stream);
    return centred ? launch_sandwich<bf16_t, true>(a, n, stream) : launch_sandwich<bf16_t, false>(a, n, stream);
}

// ---- a second embedding row, chosen by a token and the one before it --------------------------------------------

struct BigramArgs {
    float* x;                // [n, W] the stream
    const int* ids;
    const int* src;          // rows whose id the step before left in `fed`, or null
    const int* fed;
    const int* positions;
    const int* seq_of;
    const int* q_start;
    const int* q_len;
    const int* state_slots;
    int* last;               // [slots]: a request's last token
    const void* table;       // [buckets + 1, W]
    long long mul_prev, mul_cur, buckets;
    int W;
};

__device__ __forceinline__ int bigram_token(const BigramArgs& a, int t) {
    if (a.src != nullptr) {
        const int from = a.src[t];
        if (from >= 0) return a.fed[from];
    }
    return a.ids[t];
}

// A workgroup a row.  The token before a request's first row of the step is the request's state; the workgroup of that
// row is the only one that reads it, and leaves the request's last token of the step in its place.
template <typename T>
__global__ void bigram_add_kernel(BigramArgs a) {
    const int t = blockIdx.x;
    const int pos = a.positions[t];
    if (pos < 0) return;
    const int s = a.seq_of[t], start = a.q_start[s], slot = a.state_slots[s];
    if (slot < 0) return;
    const int token = bigram_token(a, t);
    long long row = a.buckets;
    if (pos > 0) {
        const long long before = t > start ? bigram_token(a, t - 1) : a.last[slot];
        row = (before * a.mul_prev + static_cast<long long>(token) * a.mul_cur) % a.buckets;
        if (row < 0) row += a.buckets;
    }
    if (t == start) {
        __syncthreads();                              // every thread has read what is replaced
        if (threadIdx.x == 0) a.last[slot] = bigram_token(a, start + a.q_len[s] - 1);
    }
    const T* add = static_cast<const T*>(a.table) + static_cast<size_t>(row) * a.W;
    float* x = a.x + static_cast<size_t>(t) * a.W;
    for (int c = threadIdx.x; c < a.W; c += blockDim.x) x[c] += to_float(add[c]);
}

extern "C" int pl_bigram_add(float* x, const int* ids, const int* src, const int* fed, const int* positions, const int* seq_of,
                             const int* q_start, const int* q_len, const int* state_slots, int* last, const void* table,
                             int dtype, long long mul_prev, long long mul_cur, long long buckets, int n, int W,
                             hipStream_t stream) {
    PL_REQUIRE(n >= 0 && W > 0 && buckets > 0, "bigram_add: %d rows of %d, %lld buckets", n, W, buckets);
    PL_REQUIRE((src == nullptr) == (fed == nullptr), "bigram_add: rows fed from the step before need both the rows and the tokens");
    if (n == 0) return 0;
    const BigramArgs a{x, ids, src, fed, positions, seq_of, q_start, q_len, state_slots, last, table, mul_prev, mul_cur, buckets, W};
    const int threads = W >= 256 ? 256 : 64;
    if (dtype == PL_DTYPE_F32) bigram_add_kernel<float><<<n, threads, 0, stream>>>(a);
    else if (dtype == PL_DTYPE_BF16) bigram_add_kernel<bf16_t><<<n, threads, 0, stream>>>(a);
    else PL_REQUIRE(false, "bigram_add: dtype code %d", dtype);
    PL_CHECK_LAUNCH("bigram_add");
    return 0;
}
