// The experts of a step of few rows (up to 64) that a router has dealt out, bfloat16 on the matrix cores: the experts' weights are
// read once, whatever the rows, and what bounds the step is that reading.  Two launches, nothing sorted in front of them:
//   up:   h[pair] = act(w_first x_row), or act(gate x) * (up x) where the experts are gated, bfloat16
//   down: y[pair] = w_down h[pair], 32-bit sums
// A workgroup of eight waves owns 32 rows of one expert's matrix (16 gate rows and their 16 up rows where gated).  It looks through the
// step's choices for the pairs that are its expert's (none: it is done), cuts the inner width into a stretch a wave,
// each wave multiplies its stretch of the weights, straight from memory in the matrix cores' layout, with its
// stretch of the pairs' rows, and the waves' sums are added in order through LDS.  A pair's result does not depend on the
// other pairs or on its place among them.
//
// D[16 x 16] += A[16 x 32] B[32 x 16], v_mfma_f32_16x16x32_bf16: lane l gives A[l % 16][8 (l / 16) ..+ 7] (a row of the weights) and
// B[8 (l / 16) ..+ 7][l % 16] (a pair's row), and holds in register r D[4 (l / 16) + r][l % 16]: four neighbouring outputs of one pair.
#include "experts.hpp"

typedef __bf16 mf_bf16x8 __attribute__((ext_vector_type(8)));
typedef float mf_f32x4 __attribute__((ext_vector_type(4)));

#define MF_WAVES 8
#define MF_ROWS 64            // rows of a step at most
#define MF_PAIRS 32           // pairs a workgroup

// One workgroup's products: up to 16 MT pairs.  `wa`, `wb`: this lane's rows of the two strips of 16 rows of the weights.  Steps of
// 32 of the inner width, U a round; a round's operands are on their way while the round before is multiplied (past the end the last step is asked
// for again, and not multiplied).
// The weights of the first MF_EARLY steps may have been asked for already (`early`).
#define MF_EARLY 2
struct FewEarly {
    mf_bf16x8 a[MF_EARLY][2];
};
__device__ __forceinline__ void few_ask_early(FewEarly& r, const bf16_t* wa, const bf16_t* wb, int first, int behind) {
#pragma unroll
    for (int u = 0; u < MF_EARLY; ++u) {
        const size_t at = static_cast<size_t>(max(min(first + u, behind - 1), 0)) * 32;
        r.a[u][0] = *reinterpret_cast<const mf_bf16x8*>(wa + at);
        r.a[u][1] = *reinterpret_cast<const mf_bf16x8*>(wb + at);
    }
}

template <int MT, int U>
struct FewRound {
    mf_bf16x8 a[U][2], x[U][MT];
};

template <int MT, int U>
__device__ __forceinline__ void few_products(const bf16_t* wa, const bf16_t* wb, const bf16_t* const (&x)[MT], int first, int behind,
                                             const FewEarly& early, mf_f32x4 (&acc)[2][MT]) {
#pragma unroll
    for (int b = 0; b < 2; ++b)
#pragma unroll
        for (int mt = 0; mt < MT; ++mt) acc[b][mt] = mf_f32x4{0.f, 0.f, 0.f, 0.f};
    if (first >= behind) return;
    auto ask_x = [&](FewRound<MT, U>& r, int k0) {
#pragma unroll
        for (int u = 0; u < U; ++u)
#pragma unroll
            for (int mt = 0; mt < MT; ++mt)
                r.x[u][mt] = *reinterpret_cast<const mf_bf16x8*>(x[mt] + static_cast<size_t>(min(k0 + u, behind - 1)) * 32);
    };
    auto ask = [&](FewRound<MT, U>& r, int k0) {
#pragma unroll
        for (int u = 0; u < U; ++u) {
            const size_t at = static_cast<size_t>(min(k0 + u, behind - 1)) * 32;
            r.a[u][0] = *reinterpret_cast<const mf_bf16x8*>(wa + at);
            r.a[u][1] = *reinterpret_cast<const mf_bf16x8*>(wb + at);
        }
        ask_x(r, k0);
    };
    auto multiply = [&](const FewRound<MT, U>& r, int k0) {
#pragma unroll
        for (int u = 0; u < U; ++u)
            if (k0 + u < behind) {                       // (the same for the whole wave)
#pragma unroll
                for (int b = 0; b < 2; ++b)
#pragma unroll
                    for (int mt = 0; mt < MT; ++mt)
                        acc[b][mt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(r.a[u][b], r.x[u][mt], acc[b][mt], 0, 0, 0);
            }
    };
    FewRound<MT, U> even, odd;
    static_assert(U <= MF_EARLY, "the first round's weights come early");
#pragma unroll
    for (int u = 0; u < U; ++u) {
        even.a[u][0] = early.a[u][0];
        even.a[u][1] = early.a[u][1];
    }
    ask_x(even, first);
    for (int k0 = first; k0 < behind; k0 += 2 * U) {
        if (k0 + U < behind) ask(odd, k0 + U);
        multiply(even, k0);
        if (k0 + U >= behind) break;
        if (k0 + 2 * U < behind) ask(even, k0 + 2 * U);
        multiply(odd, k0 + U);
    }
}

template <bool DOWN, bool GATED, int MT>
__device__ __forceinline__ void few_body(const MoeArgs& a, float* y, const bf16_t* wa, const bf16_t* wb, int N, int first, int behind,
                                         const FewEarly& early, int n0, const int* list, int pairs, mf_f32x4* red) {
    const int tid = threadIdx.x, lane = tid & 63;
    const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int c16 = lane & 15, g = lane >> 4;
    const int values = moe_row_values(a);
    constexpr bool PAIRED = GATED && !DOWN;
    const bf16_t* x[MT];
#pragma unroll
    for (int mt = 0; mt < MT; ++mt) {
        const int p = list[min(mt * 16 + c16, pairs - 1)];
        const int t = p / a.top, c = p - t * a.top;
        x[mt] = (DOWN ? static_cast<const bf16_t*>(a.h) + static_cast<size_t>(t) * values + c * a.F
                      : static_cast<const bf16_t*>(a.x) + static_cast<size_t>(t) * a.W) + 8 * g;
    }
    mf_f32x4 acc[2][MT];
    few_products<MT, MF_EARLY>(wa, wb, x, first, behind, early, acc);
    // the waves' sums, one strip after the other: [wave][mt][lane]
    mf_f32x4 sum[2];
#pragma unroll
    for (int b = 0; b < 2; ++b) {
        if (b == 1) __syncthreads();
#pragma unroll
        for (int mt = 0; mt < MT; ++mt) red[(wave * MT + mt) * 64 + lane] = acc[b][mt];
        __syncthreads();
        sum[b] = mf_f32x4{0.f, 0.f, 0.f, 0.f};
        if (tid < MT * 64) {
#pragma unroll
            for (int v = 0; v < MF_WAVES; ++v) {
                const mf_f32x4 part = red[v * MT * 64 + tid];
#pragma unroll
                for (int r = 0; r < 4; ++r) sum[b][r] += part[r];
            }
        }
    }
    const int slot = (tid >> 6) * 16 + c16;
    if (tid >= MT * 64 || slot >= pairs) return;
    const int p = list[slot];
    const int t = p / a.top, c = p - t * a.top;
#pragma unroll
    for (int b = 0; b < (PAIRED ? 1 : 2); ++b) {
        const int col = n0 + 16 * b + 4 * g;
        if (col >= N) continue;                          // (N is a multiple of 4)
        if constexpr (DOWN) {
            *reinterpret_cast<mf_f32x4*>(y + static_cast<size_t>(p) * a.W + col) = sum[b];
        } else {
            float v[4];
#pragma unroll
            for (int r = 0; r < 4; ++r)
                v[r] = PAIRED ? pl_gate_pair<false>(sum[0][r], sum[1][r], a.act, a.limit) : pl_activate<false>(sum[b][r], a.act);
            uint2 packed;
            packed.x = bf16_bits_from_float(v[0]) | (static_cast<uint32_t>(bf16_bits_from_float(v[1])) << 16);
            packed.y = bf16_bits_from_float(v[2]) | (static_cast<uint32_t>(bf16_bits_from_float(v[3])) << 16);
            *reinterpret_cast<uint2*>(static_cast<bf16_t*>(a.h) + static_cast<size_t>(t) * values + c * a.F + col) = packed;
        }
    }
}

// blockIdx.y: the expert; where there is a shared one, which has every row, it comes first.  speculate: the first weights are asked for before
// the pairs are known (most experts have some).
template <bool DOWN, bool GATED>
__global__ __launch_bounds__(64 * MF_WAVES, 4) void moe_few_kernel(MoeArgs a, float* y, int speculate) {
    __shared__ int list[MF_ROWS];
    __shared__ int wave_found[MF_WAVES];
    extern __shared__ __attribute__((aligned(16))) mf_f32x4 few_red[];
    const int group = a.shared_at < 0 ? static_cast<int>(blockIdx.y) : (blockIdx.y == 0 ? a.E : static_cast<int>(blockIdx.y) - 1);
    const bool shared = group == a.E;
    const int number = shared ? a.shared_at : group;
    const int F = shared ? a.shared_F : a.F;
    const int K = DOWN ? F : a.W, N = DOWN ? a.W : F;
    const int n0 = blockIdx.x * (GATED && !DOWN ? 16 : 32);
    if (n0 >= N) return;
    const bf16_t* w;
    if (DOWN) w = shared ? static_cast<const bf16_t*>(a.shared_down) : static_cast<const bf16_t*>(a.w_down) + static_cast<size_t>(group) * a.W * F;
    else w = shared ? static_cast<const bf16_t*>(a.shared_gu) : static_cast<const bf16_t*>(a.w_gu) + static_cast<size_t>(group) * (GATED ? 2 : 1) * F * a.W;
    const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
    const int ra = min(n0 + (lane & 15), N - 1);
    const int rb = GATED && !DOWN ? N + ra : min(n0 + 16 + (lane & 15), N - 1);
    const bf16_t* wa = w + static_cast<size_t>(ra) * K + 8 * (lane >> 4);
    const bf16_t* wb = w + static_cast<size_t>(rb) * K + 8 * (lane >> 4);
    const int chunks = K / 32, first = wave * chunks / MF_WAVES, behind = (wave + 1) * chunks / MF_WAVES;
    FewEarly early;
    const bool ahead = speculate && (blockIdx.z == 0 || shared);
    if (ahead) few_ask_early(early, wa, wb, first, behind);
    // The expert's pairs in ascending order (every workgroup of an expert has to see the same list: they take 32 pairs each).
    int found = 0;
    for (int p0 = 0; p0 < a.n * a.top; p0 += 64 * MF_WAVES) {
        const int p = p0 + threadIdx.x;
        bool mine = false;
        if (p < a.n * a.top) {
            const int t = p / a.top;
            mine = a.choice[p] == number && (!shared || p - t * a.top == a.top - 1) && a.positions[t] >= 0;
        }
        const unsigned long long mask = __ballot(mine);
        if (p0 > 0) __syncthreads();
        if (lane == 0) wave_found[wave] = __popcll(mask);
        __syncthreads();
        int at = found;
#pragma unroll
        for (int v = 0; v < MF_WAVES; ++v) {
            at += v < wave ? wave_found[v] : 0;
            found += wave_found[v];
        }
        at += __popcll(mask & ((1ull << lane) - 1ull));
        if (mine && at < MF_ROWS) list[at] = p;          // (a row names an expert once: there are no more)
    }
    __syncthreads();
    // (an expert of more than 32 pairs has a workgroup for every 32 of them: registers for twice as many would leave the chip
    // half as many waves)
    const int* mine = list + blockIdx.z * MF_PAIRS;
    const int pairs = min(min(found, MF_ROWS) - static_cast<int>(blockIdx.z) * MF_PAIRS, MF_PAIRS);
    if (pairs <= 0) return;
    if (!ahead) few_ask_early(early, wa, wb, first, behind);
    if (pairs <= 16) few_body<DOWN, GATED, 1>(a, y, wa, wb, N, first, behind, early, n0, mine, pairs, few_red);
    else few_body<DOWN, GATED, 2>(a, y, wa, wb, N, first, behind, early, n0, mine, pairs, few_red);
}

// x [n, W], the matrices and h [n, values of a row's pairs] bfloat16; y [n * top, W] 32-bit, a row a pair (a pair without an expert, and
// of an identity expert, is not written).  choice [n, top]: a row names an expert at most once.  See MoeArgs for the rest.
extern "C" int pl_moe_few(const void* x, const int* positions, const int* choice, const void* w_first, const void* w_down, void* h,
                          float* y, int n, int W, int F, int E, int top, int act, int identity, float limit, int plain, int shared_F,
                          const void* shared_first, const void* shared_down, hipStream_t stream) {
    PL_REQUIRE(n >= 0 && n <= MF_ROWS && W > 0 && F > 0 && E > 0 && E < 65535 && top > 0 && identity >= 0 && top <= E + identity + (shared_F > 0 ? 1 : 0),
               "moe_few: %d rows of %d, %d experts of %d, %d a row", n, W, E, F, top);
    PL_REQUIRE(W % 32 == 0 && F % 32 == 0 && shared_F >= 0 && shared_F % 32 == 0, "moe_few: rows of %d, experts of %d and %d (multiples of 32)", W, F, shared_F);
    PL_REQUIRE(act >= 0 && act <= (plain ? PL_ACT_RELU2 : PL_ACT_CLAMPED), "moe_few: activation code %d", act);
    PL_REQUIRE(choice != nullptr && positions != nullptr && (shared_F == 0 || (shared_first != nullptr && shared_down != nullptr)),
               "moe_few: a router's choice and the matrices of a shared expert");
    if (n == 0) return 0;
    const MoeArgs a{x, nullptr, nullptr, nullptr, positions, nullptr, w_first, w_down, h, nullptr, n, W, F, E, top, 1, act, choice, nullptr,
                    identity, limit, plain, shared_F > 0 ? E + identity : -1, shared_F, shared_first, shared_down};
    const int speculate = n * top >= 2 * E ? 1 : 0;
    const int parts = pl_ceil_div(n, MF_PAIRS);
    const int groups = E + (shared_F > 0 ? 1 : 0), widest = shared_F > F ? shared_F : F;
    const size_t lds = static_cast<size_t>(MF_WAVES) * (n <= 16 ? 1 : 2) * 64 * sizeof(mf_f32x4);
    if (plain) moe_few_kernel<false, false><<<dim3(pl_ceil_div(widest, 32), groups, parts), 64 * MF_WAVES, lds, stream>>>(a, y, speculate);
    else moe_few_kernel<false, true><<<dim3(pl_ceil_div(widest, 16), groups, parts), 64 * MF_WAVES, lds, stream>>>(a, y, speculate);
    PL_CHECK_LAUNCH("moe_few (up)");
    moe_few_kernel<true, false><<<dim3(pl_ceil_div(W, 32), groups, parts), 64 * MF_WAVES, lds, stream>>>(a, y, speculate);
    PL_CHECK_LAUNCH("moe_few (down)");
    return 0;
}
