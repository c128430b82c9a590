// The state space whose decay and step size come with the token (kind ssd of the scans): per head, with
// dt = softplus(x1 + dt_bias) and a = e^A_log,
//     S_t = e^(-a dt_t) S_(t-1) + dt_t B_t x_t^T   (N x V),     y_t = S_t^T C_t + D x_t .
// q, k and v of the scan's arguments are C, B and x; C and B have G heads, head h reads head h / (H / G).
//
// Linear attention with a fixed decay a head (kind retention) is the same recurrence with e^(-a dt) = decay, dt = 1 in front of
// B x^T and no D: the chunked kernels serve it as FIXED instances (p1 holds the decays), retention_step is its kernel for few tokens.
// Its q and k turn with their positions: retention_turn does that to a step's rows in front of the chunked kernels,
// retention_step to what it reads.
//
// ssd_step: requests of few tokens, token by token, the state read and written once, 16 bytes a lane.
//
// ssd_chunked: requests of many tokens in chunks of 64.  With b_t the sum of -a dt over a chunk's tokens up to t,
//     y_t = sum_{u<=t} e^(b_t - b_u) dt_u (C_t . B_u) x_u + e^(b_t) S_0^T C_t + D x_t ,
// so a chunk adds sum_u e^(b_L - b_u) dt_u B_u x_u^T to the state (`summary`, every chunk at once), the states
// before the chunks follow by a short walk (`carry`), and a chunk's read-outs are three small products (`output`,
// every chunk at once).  The products run on the matrix cores in 32-bit (v_mfma_f32_32x32x2_f32: 32-bit operands, 32-bit
// multiply-add).  The sums b are kept in 64-bit: decays of a chunk may be anything from 1 to 0 beside each other, what
// enters an exponential is a difference of two sums, and a small difference of large sums would lose its digits in 32.
//
// The matrix instruction, D[32 x 32] += A[32 x 2] B[2 x 32]: lane l gives A[l % 32][l / 32] and B[l / 32][l % 32]
// and holds, in register r, D[8 (r / 4) + 4 (l / 32) + r % 4][l % 32].  The order of the inner index is free as long as A and
// B agree: the two halves of a wave take runs of four, 8 q + 4 (l / 32) + e for e = 0 .. 3, so that an operand whose
// rows lie along the inner index is read 16 bytes a lane.
#include "recurrent.hpp"

typedef float ssd_f32x16 __attribute__((ext_vector_type(16)));
typedef float ssd_f32x4 __attribute__((ext_vector_type(4)));

#define SSD_CHUNK 64

__device__ __forceinline__ ssd_f32x16 ssd_mfma(float a, float b, ssd_f32x16 c) {
    return __builtin_amdgcn_mfma_f32_32x32x2f32(a, b, c, 0, 0, 0);
}

// ---- few tokens ----------------------------------------------------------------------------------------

// A workgroup of four waves owns 64 columns of a head's state for one request.  A thread holds R rows of four columns:
// rows (4 wave + lane / 16) R .. + R - 1, columns 4 (lane % 16) .. + 3.  ALIGNED: k, q and v may be read 16 bytes at a time.
template <int R, bool ALIGNED>
__global__ __launch_bounds__(256) void ssd_step_kernel(ScanArgs a) {
    __shared__ ssd_f32x4 part[4][16];
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    const int h = blockIdx.y, s = blockIdx.z;
    const int slot = a.state_slots[s];
    const int count = a.q_len[s];
    if (slot < 0 || count <= 0 || (a.below > 0 && count >= a.below)) return;
    const int start = a.q_start[s];
    const int N = a.D, V = a.V, H = a.H;
    const int g = h / (H / a.G);
    const int n0 = (4 * wave + (lane >> 4)) * R;
    const int v0 = blockIdx.x * 64 + 4 * (lane & 15);
    const bool owns = v0 < V;                                   // (V is a multiple of 4)
    float* Sg = a.state + static_cast<size_t>(slot) * a.state_stride + a.s_off + static_cast<size_t>(h) * N * V;
    ssd_f32x4 S[R];
#pragma unroll
    for (int i = 0; i < R; ++i)
        S[i] = (owns && n0 + i < N) ? *reinterpret_cast<const ssd_f32x4*>(Sg + static_cast<size_t>(n0 + i) * V + v0) : ssd_f32x4{0.f, 0.f, 0.f, 0.f};
    const float rate = expf(a.p1[h]), bias = a.p2[h], skip = a.p3[h];
    for (int t = 0; t < count; ++t) {
        const float* row = a.qkv + static_cast<size_t>(start + t) * a.qkv_stride;
        const float* kr = row + a.k_off + g * N;
        const float* qr = row + a.q_off + g * N;
        float k[R], q[R];
        if (ALIGNED && R % 4 == 0) {                            // (N is a multiple of 4 then)
#pragma unroll
            for (int i = 0; i < R; i += 4) {
                const bool in = n0 + i < N;
                const ssd_f32x4 kk = in ? *reinterpret_cast<const ssd_f32x4*>(kr + n0 + i) : ssd_f32x4{0.f, 0.f, 0.f, 0.f};
                const ssd_f32x4 qq = in ? *reinterpret_cast<const ssd_f32x4*>(qr + n0 + i) : ssd_f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    k[(i + e) % R] = kk[e];
                    q[(i + e) % R] = qq[e];
                }
            }
        } else {
#pragma unroll
            for (int i = 0; i < R; ++i) {
                k[i] = n0 + i < N ? kr[n0 + i] : 0.f;
                q[i] = n0 + i < N ? qr[n0 + i] : 0.f;
            }
        }
        ssd_f32x4 v = {0.f, 0.f, 0.f, 0.f};
        if (owns) {
            const float* vr = row + a.v_off + h * V + v0;
            if (ALIGNED) v = *reinterpret_cast<const ssd_f32x4*>(vr);
            else v = ssd_f32x4{vr[0], vr[1], vr[2], vr[3]};
        }
        const float dt = softplus_f(a.gates[static_cast<size_t>(start + t) * a.gates_stride + a.g1_off + h] + bias);
        const float keep = expf(-rate * dt);
        ssd_f32x4 o = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int i = 0; i < R; ++i) {
            const float kd = k[i] * dt;
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                S[i][e] = keep * S[i][e] + kd * v[e];
                o[e] += S[i][e] * q[i];
            }
        }
#pragma unroll
        for (int off = 16; off < 64; off <<= 1)
#pragma unroll
            for (int e = 0; e < 4; ++e) o[e] += __shfl_xor(o[e], off, 64);
        if (lane < 16) part[wave][lane] = o;
        __syncthreads();
        if (wave == 0 && lane < 16 && owns) {
            ssd_f32x4 y = part[0][lane];
#pragma unroll
            for (int w = 1; w < 4; ++w)
#pragma unroll
                for (int e = 0; e < 4; ++e) y[e] += part[w][lane][e];
#pragma unroll
            for (int e = 0; e < 4; ++e) y[e] += skip * v[e];
            *reinterpret_cast<ssd_f32x4*>(a.out + static_cast<size_t>(start + t) * (H * V) + h * V + v0) = y;
        }
        __syncthreads();
    }
#pragma unroll
    for (int i = 0; i < R; ++i)
        if (owns && n0 + i < N) *reinterpret_cast<ssd_f32x4*>(Sg + static_cast<size_t>(n0 + i) * V + v0) = S[i];
}

// How q and k of a head turn: values i and i + dims / 2 by position * freq[i], cosine and sine times `amplitude`, i < dims / 2;
// k times `k_scale` behind that.
struct HalfTurn {
    const float* freq;
    const int* positions;
    int dims;
    float amplitude, k_scale;
};

// Pair i of q and k (values i and i + dims / 2), turned.
struct TurnedPair {
    float q0, q1, k0, k1;
};
__device__ __forceinline__ TurnedPair turn_pair(const float* q, const float* k, int i, int half, float cs, float sn, float k_scale) {
    const float q0 = q[i], q1 = q[i + half], k0 = k[i], k1 = k[i + half];
    return {q0 * cs - q1 * sn, q1 * cs + q0 * sn, (k0 * cs - k1 * sn) * k_scale, (k1 * cs + k0 * sn) * k_scale};
}
__device__ __forceinline__ void half_angle(const HalfTurn& turn, int position, int i, float& cs, float& sn) {
    sincosf(static_cast<float>(position) * turn.freq[i], &sn, &cs);
    cs *= turn.amplitude;
    sn *= turn.amplitude;
}

// As ssd_step_kernel, a workgroup 64 columns of a head's state for one request; every token's q and k are turned into LDS first
// (`turns`: they have not been turned yet).
template <int R>
__global__ __launch_bounds__(256) void retention_step_kernel(ScanArgs a, HalfTurn turn, int turns) {
    __shared__ ssd_f32x4 part[4][16];
    __shared__ __attribute__((aligned(16))) float qs[16 * R], ks[16 * R];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const int h = blockIdx.y, s = blockIdx.z;
    const int slot = a.state_slots[s];
    const int count = a.q_len[s];
    if (slot < 0 || count <= 0 || (a.below > 0 && count >= a.below)) return;
    const int start = a.q_start[s];
    const int N = a.D, V = a.V, H = a.H;
    const int n0 = (4 * wave + (lane >> 4)) * R;
    const int v0 = blockIdx.x * 64 + 4 * (lane & 15);
    const bool owns = v0 < V;                                   // (V is a multiple of 4)
    float* Sg = a.state + static_cast<size_t>(slot) * a.state_stride + a.s_off + static_cast<size_t>(h) * N * V;
    ssd_f32x4 S[R];
#pragma unroll
    for (int i = 0; i < R; ++i)
        S[i] = (owns && n0 + i < N) ? *reinterpret_cast<const ssd_f32x4*>(Sg + static_cast<size_t>(n0 + i) * V + v0) : ssd_f32x4{0.f, 0.f, 0.f, 0.f};
    const float keep = a.p1[h];
    const int half = turns ? turn.dims / 2 : 0;
    const float k_scale = turns ? turn.k_scale : 1.f;
    for (int i = N + tid; i < 16 * R; i += 256) qs[i] = ks[i] = 0.f;
    for (int t = 0; t < count; ++t) {
        const float* row = a.qkv + static_cast<size_t>(start + t) * a.qkv_stride;
        const float* kr = row + a.k_off + h * N;
        const float* qr = row + a.q_off + h * N;
        ssd_f32x4 v = {0.f, 0.f, 0.f, 0.f};
        if (owns) {
            const float* vr = row + a.v_off + h * V + v0;
            v = ssd_f32x4{vr[0], vr[1], vr[2], vr[3]};
        }
        if (tid < half) {
            float cs, sn;
            half_angle(turn, turn.positions[start + t], tid, cs, sn);
            const TurnedPair p = turn_pair(qr, kr, tid, half, cs, sn, k_scale);
            qs[tid] = p.q0;
            qs[tid + half] = p.q1;
            ks[tid] = p.k0;
            ks[tid + half] = p.k1;
        } else if (tid + half < N) {
            qs[tid + half] = qr[tid + half];
            ks[tid + half] = kr[tid + half] * k_scale;
        }
        __syncthreads();
        float k[R], q[R];
#pragma unroll
        for (int i = 0; i < R; ++i) {
            k[i] = ks[n0 + i];
            q[i] = qs[n0 + i];
        }
        ssd_f32x4 o = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int i = 0; i < R; ++i)
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                S[i][e] = keep * S[i][e] + k[i] * v[e];
                o[e] += S[i][e] * q[i];
            }
#pragma unroll
        for (int off = 16; off < 64; off <<= 1)
#pragma unroll
            for (int e = 0; e < 4; ++e) o[e] += __shfl_xor(o[e], off, 64);
        if (lane < 16) part[wave][lane] = o;
        __syncthreads();
        if (wave == 0 && lane < 16 && owns) {
            ssd_f32x4 y = part[0][lane];
#pragma unroll
            for (int w = 1; w < 4; ++w)
#pragma unroll
                for (int e = 0; e < 4; ++e) y[e] += part[w][lane][e];
            *reinterpret_cast<ssd_f32x4*>(a.out + static_cast<size_t>(start + t) * (H * V) + h * V + v0) = y;
        }
        // (nobody writes `part` again before the next token's first barrier, which the first wave reaches behind its reads)
    }
#pragma unroll
    for (int i = 0; i < R; ++i)
        if (owns && n0 + i < N) *reinterpret_cast<ssd_f32x4*>(Sg + static_cast<size_t>(n0 + i) * V + v0) = S[i];
}

// A workgroup a token: q and k of every head, turned in place.
__global__ __launch_bounds__(256) void retention_turn_kernel(float* __restrict__ rows, int stride, int q_off, int k_off, int H, int N, HalfTurn turn) {
    __shared__ float cosine[128], sine[128];
    const int t = blockIdx.x;
    const int position = turn.positions[t];
    if (position < 0) return;
    const int half = turn.dims / 2, each = N - half;             // pairs, then the values that do not turn
    for (int i = threadIdx.x; i < half; i += 256) half_angle(turn, position, i, cosine[i], sine[i]);
    __syncthreads();
    float* row = rows + static_cast<size_t>(t) * stride;
    for (int e = threadIdx.x; e < H * each; e += 256) {
        const int h = e / each, i = e - h * each;
        float* q = row + q_off + h * N;
        float* k = row + k_off + h * N;
        if (i < half) {
            const TurnedPair p = turn_pair(q, k, i, half, cosine[i], sine[i], turn.k_scale);
            q[i] = p.q0;
            q[i + half] = p.q1;
            k[i] = p.k0;
            k[i + half] = p.k1;
        } else {
            k[i + half] *= turn.k_scale;
        }
    }
}

// ---- many tokens -----------------------------------------------------------------------------------------

struct SsdArgs {
    ScanArgs a;
    float* U;        // [chunks, H, N, V]  a chunk's weighted sum of B x^T
    float* Sin;      // [chunks, H, N, V]  the state before a chunk
    float* ends;     // [chunks, H]        b at the chunk's end
};

// A request's chunks have numbers of their own among all chunks of the step: requests lie one behind the
// other in the step's rows, so q_start / 64 + (index of the request) + (chunk in the request) is unique.
__device__ __forceinline__ int ssd_chunk(const ScanArgs& a, int s, int c) { return a.q_start[s] / SSD_CHUNK + s + c; }

// By one wave, all its lanes: the running sums b (64-bit) and the step sizes of a chunk's L <= 64 tokens; the sum
// over the chunk comes back.  Lanes past the chunk hold the last sum and a step of zero.
template <bool FIXED>
__device__ __forceinline__ double ssd_gates(const ScanArgs& a, int h, int row0, int L, int lane, double& b, float& dt) {
    dt = 0.f;
    if (FIXED) {
        const double each = log(static_cast<double>(a.p1[h]));
        if (lane < L) dt = 1.f;
        b = each * (min(lane, L - 1) + 1);
        return each * L;
    }
    if (lane < L) dt = softplus_f(a.gates[static_cast<size_t>(row0 + lane) * a.gates_stride + a.g1_off + h] + a.p2[h]);
    double sum = -static_cast<double>(expf(a.p1[h])) * static_cast<double>(dt);
#pragma unroll
    for (int off = 1; off < 64; off <<= 1) {
        const double other = __shfl_up(sum, off, 64);
        if (lane >= off) sum += other;
    }
    b = sum;
    return __shfl(sum, L - 1, 64);
}

// (FIXED: one decay a head, p1, and steps of one.)

// summary: a wave a tile of 32 rows of N (and the tile four further on, where N has more than 128), 64 columns of V.
// Both operands come straight from memory, a token a row: 128 bytes a half wave.
template <bool FIXED>
__global__ __launch_bounds__(256) void ssd_summary_kernel(SsdArgs sa) {
    const ScanArgs& a = sa.a;
    __shared__ float weight[SSD_CHUNK];
    const int N = a.D, V = a.V, H = a.H;
    const int tiles = (V + 63) / 64;
    const int c = blockIdx.x, h = blockIdx.y / tiles, vt = blockIdx.y % tiles, s = blockIdx.z;
    const int slot = a.state_slots[s], count = a.q_len[s];
    if (slot < 0 || count < a.below || c * SSD_CHUNK >= count) return;
    const int L = min(SSD_CHUNK, count - c * SSD_CHUNK), row0 = a.q_start[s] + c * SSD_CHUNK;
    const size_t idx = static_cast<size_t>(ssd_chunk(a, s, c)) * H + h;
    const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
    const int l32 = lane & 31, half = lane >> 5;
    const int g = h / (H / a.G);
    const bool two = vt * 64 + 32 < V;               // whether the second 32 columns exist
    const int va = min(vt * 64 + l32, V - 1), vb = min(vt * 64 + 32 + l32, V - 1);
    float xa[SSD_CHUNK / 2], xb[SSD_CHUNK / 2];
    const float* rows = a.qkv + static_cast<size_t>(row0) * a.qkv_stride;
#pragma unroll
    for (int k = 0; k < SSD_CHUNK / 2; ++k) {
        const float* x = rows + static_cast<size_t>(min(2 * k + half, L - 1)) * a.qkv_stride + a.v_off + h * V;
        xa[k] = x[va];
        xb[k] = two ? x[vb] : 0.f;
    }
    if (wave == 0) {
        double b;
        float dt;
        const double end = ssd_gates<FIXED>(a, h, row0, L, lane, b, dt);
        weight[lane] = expf(static_cast<float>(end - b)) * dt;          // (zero past the chunk's tokens)
        if (vt == 0 && lane == 0) sa.ends[idx] = static_cast<float>(end);
    }
    __syncthreads();
#pragma unroll
    for (int k = 0; k < SSD_CHUNK / 2; ++k) {
        const float w = weight[2 * k + half];
        xa[k] *= w;
        xb[k] *= w;
    }
    float* U = sa.U + idx * N * V;
    for (int n0 = wave * 32; n0 < N; n0 += 128) {
        const int n = min(n0 + l32, N - 1);
        float ka[SSD_CHUNK / 2];
#pragma unroll
        for (int k = 0; k < SSD_CHUNK / 2; ++k)
            ka[k] = rows[static_cast<size_t>(min(2 * k + half, L - 1)) * a.qkv_stride + a.k_off + g * N + n];
        ssd_f32x16 da, db;
#pragma unroll
        for (int r = 0; r < 16; ++r) da[r] = db[r] = 0.f;
#pragma unroll
        for (int k = 0; k < SSD_CHUNK / 2; ++k) {
            da = ssd_mfma(ka[k], xa[k], da);
            if (two) db = ssd_mfma(ka[k], xb[k], db);
        }
#pragma unroll
        for (int r = 0; r < 16; ++r) {
            const int row = n0 + 8 * (r >> 2) + 4 * half + (r & 3);
            if (row >= N) continue;
            if (vt * 64 + l32 < V) U[static_cast<size_t>(row) * V + vt * 64 + l32] = da[r];
            if (vt * 64 + 32 + l32 < V) U[static_cast<size_t>(row) * V + vt * 64 + 32 + l32] = db[r];
        }
    }
}

// carry: the state before every chunk, and the request's state after its last; a thread an element, the sums of the next
// chunks on their way while the ones before are taken in.
__global__ __launch_bounds__(256) void ssd_carry_kernel(SsdArgs sa) {
    const ScanArgs& a = sa.a;
    const int N = a.D, V = a.V, H = a.H;
    const int h = blockIdx.y, s = blockIdx.z;
    const int slot = a.state_slots[s], count = a.q_len[s];
    if (slot < 0 || count < a.below) return;
    const int chunks = (count + SSD_CHUNK - 1) / SSD_CHUNK;
    const int e = blockIdx.x * 256 + threadIdx.x;
    if (e >= N * V) return;
    const size_t NV = static_cast<size_t>(N) * V;
    float* at = a.state + static_cast<size_t>(slot) * a.state_stride + a.s_off + h * NV + e;
    const size_t first = static_cast<size_t>(ssd_chunk(a, s, 0)) * H + h;
    const float* __restrict__ U = sa.U + first * NV + e;
    float* __restrict__ Sin = sa.Sin + first * NV + e;
    const float* __restrict__ ends = sa.ends + first;
    const size_t step = NV * H;
    float S = *at;
    constexpr int AHEAD = 8;
    for (int c0 = 0; c0 < chunks; c0 += AHEAD) {
        float u[AHEAD], keep[AHEAD];
#pragma unroll
        for (int i = 0; i < AHEAD; ++i) {
            const int c = min(c0 + i, chunks - 1);
            u[i] = U[c * step];
            keep[i] = ends[static_cast<size_t>(c) * H];
        }
#pragma unroll
        for (int i = 0; i < AHEAD; ++i)
            if (c0 + i < chunks) {
                Sin[(c0 + i) * step] = S;
                S = expf(keep[i]) * S + u[i];
            }
    }
    *at = S;
}

// output: the read-outs of one chunk, head and tile of 64 columns.  Four waves; wave 2 ti + j owns the tokens 32 ti .. + 31 and, of the
// scores, the earlier tokens 32 j .. + 31, of the read-outs, the columns 32 j .. + 31.
// LDS: C [64][P], B [64][P] (behind the scores' barrier the weighted scores [64][68] lie in its place), b, step sizes.
template <bool FIXED>
__global__ __launch_bounds__(256, 2) void ssd_output_kernel(SsdArgs sa, int aligned) {
    const ScanArgs& a = sa.a;
    extern __shared__ __attribute__((aligned(16))) float lds[];
    const int N = a.D, V = a.V, H = a.H;
    const int tiles = (V + 63) / 64;
    const int c = blockIdx.x, h = blockIdx.y / tiles, vt = blockIdx.y % tiles, s = blockIdx.z;
    const int slot = a.state_slots[s], count = a.q_len[s];
    if (slot < 0 || count < a.below || c * SSD_CHUNK >= count) return;
    const int L = min(SSD_CHUNK, count - c * SSD_CHUNK), row0 = a.q_start[s] + c * SSD_CHUNK;
    const size_t idx = static_cast<size_t>(ssd_chunk(a, s, c)) * H + h;
    const int g = h / (H / a.G);
    const int Np = (N + 7) & ~7, P = Np + 4;
    constexpr int PA = SSD_CHUNK + 4;
    double* bd = reinterpret_cast<double*>(lds);
    float* dts = lds + 2 * SSD_CHUNK;
    float* Cs = dts + SSD_CHUNK;
    float* Bs = Cs + SSD_CHUNK * P;
    float* As = Bs;
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int l32 = lane & 31, half = lane >> 5;
    const int ti = wave >> 1, tj = wave & 1;
    const float* rows = a.qkv + static_cast<size_t>(row0) * a.qkv_stride;

    // ---- what waits for nothing: C and B into LDS, the columns of x into registers, the first rows of S_0 ----
    if (aligned) {
        const int quads = Np / 4;
        for (int e = tid; e < SSD_CHUNK * quads; e += 256) {
            const int t = e / quads, i = 4 * (e - t * quads);
            ssd_f32x4 cv = {0.f, 0.f, 0.f, 0.f}, bv = cv;
            if (t < L && i < N) {
                const float* row = rows + static_cast<size_t>(t) * a.qkv_stride + g * N + i;
                cv = *reinterpret_cast<const ssd_f32x4*>(row + a.q_off);
                bv = *reinterpret_cast<const ssd_f32x4*>(row + a.k_off);
            }
            *reinterpret_cast<ssd_f32x4*>(Cs + t * P + i) = cv;
            *reinterpret_cast<ssd_f32x4*>(Bs + t * P + i) = bv;
        }
    } else {
        for (int e = tid; e < SSD_CHUNK * Np; e += 256) {
            const int t = e / Np, i = e - t * Np;
            const bool in = t < L && i < N;
            const float* row = rows + static_cast<size_t>(in ? t : 0) * a.qkv_stride + g * N + (in ? i : 0);
            Cs[t * P + i] = in ? row[a.q_off] : 0.f;
            Bs[t * P + i] = in ? row[a.k_off] : 0.f;
        }
    }
    const int v = vt * 64 + 32 * tj + l32, vc = min(v, V - 1);
    const bool columns = vt * 64 + 32 * tj < V && 32 * ti < L;      // (the same for the wave) it has read-outs to give
    float x[SSD_CHUNK / 2];                                           // x of token 8 q + 4 half + e in x[4 q + e]
#pragma unroll
    for (int k = 0; k < SSD_CHUNK / 2; ++k) {
        x[k] = 0.f;
        if (columns && (k < 16 || ti == 1)) {
            const int u = 8 * (k >> 2) + 4 * half + (k & 3);
            x[k] = rows[static_cast<size_t>(min(u, L - 1)) * a.qkv_stride + a.v_off + h * V + vc];
        }
    }
    const float* S0 = sa.Sin + idx * N * V + vc;
    auto ask = [&](int n0, float (&s0)[32]) {                         // rows n0 .. n0 + 63 of S_0, the wave's columns
#pragma unroll
        for (int k = 0; k < 32; ++k) {
            const int n = n0 + 8 * (k >> 2) + 4 * half + (k & 3);
            s0[k] = S0[static_cast<size_t>(min(n, N - 1)) * V];
        }
    };
    float s0[32];
    if (columns) ask(0, s0);
    if (wave == 0) {
        double b;
        float dt;
        ssd_gates<FIXED>(a, h, row0, L, lane, b, dt);
        bd[lane] = b;
        dts[lane] = dt;
    }
    __syncthreads();

    // ---- the scores C_t . B_u of a tile of 32 by 32 (the tile of later tokens against earlier ones is all hidden) ----
    const bool scored = tj <= ti && 32 * ti < L;
    ssd_f32x16 acc;
#pragma unroll
    for (int r = 0; r < 16; ++r) acc[r] = 0.f;
    if (scored) {
        const float* ca = Cs + (32 * ti + l32) * P + 4 * half;
        const float* ba = Bs + (32 * tj + l32) * P + 4 * half;
        for (int q = 0; q < Np; q += 8) {
            const ssd_f32x4 cv = *reinterpret_cast<const ssd_f32x4*>(ca + q), bv = *reinterpret_cast<const ssd_f32x4*>(ba + q);
#pragma unroll
            for (int e = 0; e < 4; ++e) acc = ssd_mfma(cv[e], bv[e], acc);
        }
        const int u = 32 * tj + l32;
        const double bu = bd[u];
        const float du = dts[u];
#pragma unroll
        for (int r = 0; r < 16; ++r) {
            const int t = 32 * ti + 8 * (r >> 2) + 4 * half + (r & 3);
            acc[r] = (u <= t && t < L) ? acc[r] * (expf(static_cast<float>(bd[t] - bu)) * du) : 0.f;
        }
    }
    __syncthreads();                                                  // nobody reads B any more
    if (scored) {
#pragma unroll
        for (int r = 0; r < 16; ++r) As[(32 * ti + 8 * (r >> 2) + 4 * half + (r & 3)) * PA + 32 * tj + l32] = acc[r];
    }
    // ---- S_0^T C_t, times e^(b_t) ----
    ssd_f32x16 y;
#pragma unroll
    for (int r = 0; r < 16; ++r) y[r] = 0.f;
    if (columns) {
        const float* ca = Cs + (32 * ti + l32) * P + 4 * half;
        for (int n0 = 0; n0 < Np; n0 += 64) {
            float now[32];
#pragma unroll
            for (int k = 0; k < 32; ++k) now[k] = s0[k];
            if (n0 + 64 < Np) ask(n0 + 64, s0);
#pragma unroll
            for (int q = 0; q < 8; ++q) {
                if (n0 + 8 * q < Np) {
                    const ssd_f32x4 cv = *reinterpret_cast<const ssd_f32x4*>(ca + n0 + 8 * q);   // (zeros past N)
#pragma unroll
                    for (int e = 0; e < 4; ++e) y = ssd_mfma(cv[e], now[4 * q + e], y);
                }
            }
        }
#pragma unroll
        for (int r = 0; r < 16; ++r) y[r] *= expf(static_cast<float>(bd[32 * ti + 8 * (r >> 2) + 4 * half + (r & 3)]));
    }
    __syncthreads();                                                  // the weighted scores are written
    if (!columns) return;
    // ---- the weighted scores times x, and D x ----
    {
        const float* sc = As + (32 * ti + l32) * PA + 4 * half;
#pragma unroll
        for (int q = 0; q < 8; ++q) {
            if (q < 4 || ti == 1) {
                const ssd_f32x4 av = *reinterpret_cast<const ssd_f32x4*>(sc + 8 * q);
#pragma unroll
                for (int e = 0; e < 4; ++e) y = ssd_mfma(av[e], x[4 * q + e], y);
            }
        }
    }
    const float skip = FIXED ? 0.f : a.p3[h];
    float* out = a.out + static_cast<size_t>(row0) * (H * V) + h * V;
#pragma unroll
    for (int r = 0; r < 16; ++r) {
        const int t = 32 * ti + 8 * (r >> 2) + 4 * half + (r & 3);
        // (token t's own x is the one this lane holds in the same place of its half of the chunk)
        if (t < L && v < V) out[static_cast<size_t>(t) * (H * V) + v] = FIXED ? y[r] : y[r] + skip * (ti == 0 ? x[r] : x[16 + r]);
    }
}

static bool ssd_aligned(const ScanArgs& a) {
    return ((a.qkv_stride | a.q_off | a.k_off | a.v_off | a.D) & 3) == 0 && reinterpret_cast<uintptr_t>(a.qkv) % 16 == 0;
}

// Whether ssd_step serves a state of V columns with slots `state_stride` floats apart (the scan kernel does otherwise).
extern "C" int pl_ssd_step_applies(int V, long state_stride) { return V % 4 == 0 && state_stride % 4 == 0 ? 1 : 0; }

// The requests that bring fewer than `below` tokens (0: all), token by token.
extern "C" int pl_ssd_step(const float* qkv, int qkv_stride, int q_off, int k_off, int v_off, const float* gates, int gates_stride,
                           int g_off, const float* a_log, const float* dt_bias, const float* skip, float* state, long state_stride,
                           float* out, const int* q_start, const int* q_len, const int* state_slots, int seqs, int H, int G, int N,
                           int V, int below, hipStream_t stream) {
    PL_REQUIRE(H > 0 && G > 0 && H % G == 0 && H <= 65535 && seqs >= 0 && seqs <= 65535, "ssd_step: %d heads over %d groups, %d requests", H, G, seqs);
    PL_REQUIRE(N > 0 && N <= 256 && V > 0 && pl_ssd_step_applies(V, state_stride) && reinterpret_cast<uintptr_t>(state) % 16 == 0 &&
               reinterpret_cast<uintptr_t>(out) % 16 == 0, "ssd_step: a state of %d by %d a head, slots of %ld floats", N, V, state_stride);
    PL_REQUIRE(gates != nullptr && a_log != nullptr && dt_bias != nullptr && skip != nullptr, "ssd_step: constants of the heads are missing");
    if (seqs == 0) return 0;
    const ScanArgs a{qkv, qkv_stride, q_off, k_off, v_off, gates, gates_stride, g_off, 0, a_log, dt_bias, skip, 0.f, state, state_stride,
                     0, 0, 0, out, q_start, q_len, state_slots, H, G, N, V, below};
    const dim3 grid(pl_ceil_div(V, 64), H, seqs);
    const bool aligned = ssd_aligned(a);
#define SSD_STEP(R)                                                              \
    do {                                                                         \
        if (aligned) ssd_step_kernel<R, true><<<grid, 256, 0, stream>>>(a);      \
        else ssd_step_kernel<R, false><<<grid, 256, 0, stream>>>(a);             \
    } while (0)
    if (N <= 16) SSD_STEP(1);
    else if (N <= 32) SSD_STEP(2);
    else if (N <= 64) SSD_STEP(4);
    else if (N <= 128) SSD_STEP(8);
    else SSD_STEP(16);
#undef SSD_STEP
    PL_CHECK_LAUNCH("ssd_step");
    return 0;
}

template <bool FIXED>
static int launch_chunks(const SsdArgs& sa, int seqs, int max_q_len, hipStream_t stream) {
    const ScanArgs& a = sa.a;
    const int N = a.D, V = a.V, tiles = pl_ceil_div(V, 64);
    const dim3 grid(pl_ceil_div(max_q_len, SSD_CHUNK), a.H * tiles, seqs);
    ssd_summary_kernel<FIXED><<<grid, 256, 0, stream>>>(sa);
    PL_CHECK_LAUNCH("ssd_chunked (summary)");
    ssd_carry_kernel<<<dim3(pl_ceil_div(N * V, 256), a.H, seqs), 256, 0, stream>>>(sa);
    PL_CHECK_LAUNCH("ssd_chunked (carry)");
    const int P = ((N + 7) & ~7) + 4;
    const size_t lds = (3 * SSD_CHUNK + SSD_CHUNK * static_cast<size_t>(P) + SSD_CHUNK * static_cast<size_t>(P > SSD_CHUNK + 4 ? P : SSD_CHUNK + 4)) * sizeof(float);
    if (lds > 48 * 1024) {
        hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void*>(&ssd_output_kernel<FIXED>), hipFuncAttributeMaxDynamicSharedMemorySize, static_cast<int>(lds));
        PL_REQUIRE(e == hipSuccess, "ssd_chunked: %zu bytes of LDS refused: %s", lds, hipGetErrorString(e));
    }
    ssd_output_kernel<FIXED><<<grid, 256, lds, stream>>>(sa, ssd_aligned(a) ? 1 : 0);
    PL_CHECK_LAUNCH("ssd_chunked (output)");
    return 0;
}

// The requests that bring at least `from` tokens, in chunks of 64.  U, Sin: room for (rows / 64 + requests + 1) chunks of
// H * N * V floats; ends: of H.
extern "C" int pl_ssd_chunked(const float* qkv, int qkv_stride, int q_off, int k_off, int v_off, const float* gates, int gates_stride,
                              int g_off, const float* a_log, const float* dt_bias, const float* skip, float* state, long state_stride,
                              float* out, const int* q_start, const int* q_len, const int* state_slots, int seqs, int max_q_len, int H,
                              int G, int N, int V, int from, float* U, float* Sin, float* ends, hipStream_t stream) {
    PL_REQUIRE(H > 0 && G > 0 && H % G == 0 && N > 0 && N <= 256 && V > 0 && from >= 1, "ssd_chunked: %d heads of %d by %d over %d groups, from %d tokens", H, N, V, G, from);
    PL_REQUIRE(gates != nullptr && a_log != nullptr && dt_bias != nullptr && skip != nullptr && U != nullptr && Sin != nullptr && ends != nullptr,
               "ssd_chunked: constants of the heads or room for the chunks' sums are missing");
    const int tiles = pl_ceil_div(V, 64);
    PL_REQUIRE(static_cast<long long>(H) * tiles <= 65535 && seqs >= 0 && seqs <= 65535, "ssd_chunked: %d heads of %d columns, %d requests", H, V, seqs);
    if (seqs == 0 || max_q_len < from) return 0;
    const SsdArgs sa{{qkv, qkv_stride, q_off, k_off, v_off, gates, gates_stride, g_off, 0, a_log, dt_bias, skip, 0.f, state, state_stride,
                      0, 0, 0, out, q_start, q_len, state_slots, H, G, N, V, from}, U, Sin, ends};
    return launch_chunks<false>(sa, seqs, max_q_len, stream);
}

// Retention: S = decay S + k v^T, o = S^T q, q and k turning with their positions (HalfTurn; freq null: not at all).
// The rows of q and k in `rows` turn in place.
extern "C" int pl_retention_turn(float* rows, int stride, int q_off, int k_off, int n, int H, int N, const float* freq, int dims,
                                 float amplitude, float k_scale, const int* positions, hipStream_t stream) {
    PL_REQUIRE(n >= 0 && H > 0 && N > 0 && N <= 256 && dims >= 0 && dims % 2 == 0 && dims <= N && (dims == 0 || freq != nullptr) && positions != nullptr,
               "retention_turn: %d heads of %d values, %d of which turn", H, N, dims);
    PL_REQUIRE(q_off >= 0 && k_off >= 0 && q_off + H * N <= stride && k_off + H * N <= stride, "retention_turn: q and k at %d and %d of rows of %d", q_off, k_off, stride);
    if (n == 0) return 0;
    retention_turn_kernel<<<n, 256, 0, stream>>>(rows, stride, q_off, k_off, H, N, HalfTurn{freq, positions, dims, amplitude, k_scale});
    PL_CHECK_LAUNCH("retention_turn");
    return 0;
}

// The requests that bring fewer than `below` tokens (0: all), token by token.  turns: q and k of these rows have not been turned.
extern "C" int pl_retention_step(const float* qkv, int qkv_stride, int q_off, int k_off, int v_off, const float* decay, const float* freq,
                                 int dims, float amplitude, float k_scale, int turns, const int* positions, float* state, long state_stride,
                                 float* out, const int* q_start, const int* q_len, const int* state_slots, int seqs, int H, int N, int V,
                                 int below, hipStream_t stream) {
    PL_REQUIRE(H > 0 && H <= 65535 && seqs >= 0 && seqs <= 65535, "retention_step: %d heads, %d requests", H, seqs);
    PL_REQUIRE(N > 0 && N <= 256 && V > 0 && pl_ssd_step_applies(V, state_stride) && reinterpret_cast<uintptr_t>(state) % 16 == 0 &&
               reinterpret_cast<uintptr_t>(out) % 16 == 0, "retention_step: a state of %d by %d a head, slots of %ld floats", N, V, state_stride);
    PL_REQUIRE(decay != nullptr && positions != nullptr && dims >= 0 && dims % 2 == 0 && dims <= N && (dims == 0 || freq != nullptr),
               "retention_step: %d of %d values turn", dims, N);
    if (seqs == 0) return 0;
    const ScanArgs a{qkv, qkv_stride, q_off, k_off, v_off, nullptr, 0, 0, 0, decay, nullptr, nullptr, 0.f, state, state_stride,
                     0, 0, 0, out, q_start, q_len, state_slots, H, H, N, V, below};
    const HalfTurn turn{freq, positions, dims, amplitude, k_scale};
    const dim3 grid(pl_ceil_div(V, 64), H, seqs);
    if (N <= 16) retention_step_kernel<1><<<grid, 256, 0, stream>>>(a, turn, turns);
    else if (N <= 32) retention_step_kernel<2><<<grid, 256, 0, stream>>>(a, turn, turns);
    else if (N <= 64) retention_step_kernel<4><<<grid, 256, 0, stream>>>(a, turn, turns);
    else if (N <= 128) retention_step_kernel<8><<<grid, 256, 0, stream>>>(a, turn, turns);
    else retention_step_kernel<16><<<grid, 256, 0, stream>>>(a, turn, turns);
    PL_CHECK_LAUNCH("retention_step");
    return 0;
}

// The requests that bring at least `from` tokens, in chunks of 64, q and k turned already; decays above zero.  Room as in pl_ssd_chunked.
extern "C" int pl_retention_chunked(const float* qkv, int qkv_stride, int q_off, int k_off, int v_off, const float* decay, float* state,
                                    long state_stride, float* out, const int* q_start, const int* q_len, const int* state_slots, int seqs,
                                    int max_q_len, int H, int N, int V, int from, float* U, float* Sin, float* ends, hipStream_t stream) {
    PL_REQUIRE(H > 0 && N > 0 && N <= 256 && V > 0 && from >= 1, "retention_chunked: %d heads of %d by %d, from %d tokens", H, N, V, from);
    PL_REQUIRE(decay != nullptr && U != nullptr && Sin != nullptr && ends != nullptr, "retention_chunked: the decays or room for the chunks' sums are missing");
    PL_REQUIRE(static_cast<long long>(H) * pl_ceil_div(V, 64) <= 65535 && seqs >= 0 && seqs <= 65535, "retention_chunked: %d heads of %d columns, %d requests", H, V, seqs);
    if (seqs == 0 || max_q_len < from) return 0;
    const SsdArgs sa{{qkv, qkv_stride, q_off, k_off, v_off, nullptr, 0, 0, 0, decay, nullptr, nullptr, 0.f, state, state_stride,
                      0, 0, 0, out, q_start, q_len, state_slots, H, H, N, V, from}, U, Sin, ends};
    return launch_chunks<true>(sa, seqs, max_q_len, stream);
}
