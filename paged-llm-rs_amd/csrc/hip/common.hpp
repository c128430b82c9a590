// Shared by every kernel file: element types, conversions, wave reductions and
// the error channel of the C interface.
#pragma once

#include <hip/hip_runtime.h>
#include <stdint.h>

#define PL_DTYPE_F32 0
#define PL_DTYPE_BF16 1

#define PL_WAVE 64

// bfloat16 as its sixteen bits.
struct bf16_t {
    uint16_t bits;
};

__device__ __forceinline__ float to_float(float x) { return x; }
__device__ __forceinline__ float to_float(bf16_t x) {
    return __uint_as_float(static_cast<uint32_t>(x.bits) << 16);
}

// Round-to-nearest-even through the hardware's conversion (v_cvt_pk_bf16_f32); a NaN stays a NaN.
__device__ __forceinline__ uint16_t bf16_bits_from_float(float f) {
    return __builtin_bit_cast(uint16_t, static_cast<__bf16>(f));
}

template <typename T>
__device__ __forceinline__ T from_float(float f);
template <>
__device__ __forceinline__ float from_float<float>(float f) {
    return f;
}
template <>
__device__ __forceinline__ bf16_t from_float<bf16_t>(float f) {
    bf16_t r;
    r.bits = bf16_bits_from_float(f);
    return r;
}

// A value of one of two element types chosen at run time (norm gains may be
// stored wider than the activations).
__device__ __forceinline__ float load_as_float(const void* p, int dtype, size_t i) {
    return dtype == PL_DTYPE_F32 ? static_cast<const float*>(p)[i]
                                 : to_float(static_cast<const bf16_t*>(p)[i]);
}

__device__ __forceinline__ float wave_sum(float v) {
#pragma unroll
    for (int off = PL_WAVE / 2; off > 0; off >>= 1) v += __shfl_xor(v, off, PL_WAVE);
    return v;
}

__device__ __forceinline__ float wave_max(float v) {
#pragma unroll
    for (int off = PL_WAVE / 2; off > 0; off >>= 1) v = fmaxf(v, __shfl_xor(v, off, PL_WAVE));
    return v;
}

// Sum over a workgroup of up to 1024 threads; every thread gets the result.
// The order of the additions is fixed by the thread layout alone.
__device__ __forceinline__ float block_sum(float v, float* scratch /* >= 16 floats of LDS */) {
    const int lane = threadIdx.x % PL_WAVE;
    const int wave = threadIdx.x / PL_WAVE;
    const int waves = (blockDim.x + PL_WAVE - 1) / PL_WAVE;
    v = wave_sum(v);
    __syncthreads();
    if (lane == 0) scratch[wave] = v;
    __syncthreads();
    float total = 0.f;
    for (int w = 0; w < waves; ++w) total += scratch[w];
    return total;
}

// ---- the activation of a gated feed-forward's gate branch ------------------------
#define PL_ACT_SILU 0
#define PL_ACT_GELU_TANH 1
#define PL_ACT_GELU 2
#define PL_ACT_RELU2 3        // max(x, 0)^2
// What a gated feed-forward may do to gate and up together instead of act(gate) * up (pl_gate_pair alone takes it):
// with g = min(gate, limit) and u = max(min(up, limit), -limit), g sigmoid(1.702 g) (u + 1).
#define PL_ACT_CLAMPED 4

// EXACT: the library's exponential (what the 32-bit path needs); otherwise the hardware's.  `act` is the
// same for a whole launch.
template <bool EXACT>
__device__ __forceinline__ float pl_activate(float g, int act) {
    if (act == PL_ACT_SILU) return g / (1.f + (EXACT ? expf(-g) : __expf(-g)));
    if (act == PL_ACT_GELU_TANH) return 0.5f * g * (1.f + tanhf(0.7978845608028654f * (g + 0.044715f * g * g * g)));
    if (act == PL_ACT_RELU2) {
        const float r = fmaxf(g, 0.f);
        return r * r;
    }
    return 0.5f * g * (1.f + erff(g * 0.7071067811865476f));
}

// What stands between the products of a gated feed-forward: act(gate) * up, or the clamped pair of PL_ACT_CLAMPED.
template <bool EXACT>
__device__ __forceinline__ float pl_gate_pair(float gate, float up, int act, float limit) {
    if (act == PL_ACT_CLAMPED) {
        const float g = fminf(gate, limit), u = fmaxf(fminf(up, limit), -limit);
        const float e = EXACT ? expf(-1.702f * g) : __expf(-1.702f * g);
        return g / (1.f + e) * (u + 1.f);
    }
    return pl_activate<EXACT>(gate, act) * up;
}

// ---- the error channel -------------------------------------------------------
// Launchers return 0 or a negative code and leave a message for pl_last_error().
void pl_set_error(const char* fmt, ...);

// The compute units of the current device (launch-size choices go by it).
int pl_compute_units();

#define PL_REQUIRE(cond, ...)            \
    do {                                 \
        if (!(cond)) {                   \
            pl_set_error(__VA_ARGS__);   \
            return -1;                   \
        }                                \
    } while (0)

#define PL_CHECK_LAUNCH(name)                                                   \
    do {                                                                        \
        hipError_t e_ = hipGetLastError();                                      \
        if (e_ != hipSuccess) {                                                 \
            pl_set_error("%s: launch failed: %s", name, hipGetErrorString(e_)); \
            return -2;                                                          \
        }                                                                       \
    } while (0)

__host__ __device__ static inline int pl_ceil_div(int a, int b) { return (a + b - 1) / b; }

// Which keys at or before its own position a query sees, as one number (the attention kernels' `window`):
// 0 all of them; w > 0 a window, its own key and the w - 1 before it; -c < 0 blocks of c positions counted
// from position 0 of the request, the keys of the query's own block.  The first key the query at `pos` sees:
__host__ __device__ static inline int pl_first_visible(int pos, int window) {
    if (window > 0) return pos + 1 > window ? pos + 1 - window : 0;
    if (window < 0) return pos - pos % (-window);
    return 0;
}

// What an attention layer may have beside its mask, its sinks and its distance slopes; all off by default.
struct PlAttentionMore {
    float cap;            // > 0: a scaled score s becomes cap * tanh(s / cap), before the distance penalty
    int keep;             // the keys 0 .. keep - 1 of a request are seen by every later query, whatever the window
    const float* gate;    // [rows, gate_stride]: head h's read-out of row t times sigmoid(gate[t, h]); null: none
    int gate_stride;
};

static inline bool pl_has_more(const PlAttentionMore& m) { return m.cap > 0.f || m.keep > 0 || m.gate != nullptr; }

__device__ __forceinline__ float pl_head_gate(const PlAttentionMore& m, int row, int head) {
    return 1.f / (1.f + expf(-m.gate[static_cast<size_t>(row) * m.gate_stride + head]));
}
