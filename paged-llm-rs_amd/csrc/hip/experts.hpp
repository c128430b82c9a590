// Shared by the kernels that run a step's rows through their experts: what a launch is told, and which expert a (row, choice)
// pair belongs to.
#pragma once

#include "common.hpp"

// The id of row t: its own, or the one an earlier kernel left on the device (as the embedding takes it).
__device__ __forceinline__ int moe_token(const int* ids, const int* src, const int* fed, int t) {
    int id = ids[t];
    if (src != nullptr) {
        const int from = src[t];
        if (from >= 0) id = fed[from];
    }
    return id;
}

struct MoeArgs {
    const void* x;         // [n, W]
    const int* ids;
    const int* src;
    const int* fed;
    const int* positions;  // rows at position -1 are padding
    const int* table;      // [vocab, top]
    const void* w_gu;      // [E, 2 F, W]: an expert's gate rows, then its up rows
    const void* w_down;    // [E, W, F]
    void* h;               // [n, top, F]
    float* out;            // [n, W]
    int n, W, F, E, top, vocab, act;
    // Where a router has chosen (null: the table decides and every choice counts 1/top): the expert of pair
    // (t, c) is choice[t * top + c], -1 for none, E .. E + identity - 1 for an identity expert, whose output is the
    // row itself; weight[t * top + c] is what the pair counts.
    const int* choice;
    const float* weight;
    int identity;
    float limit;           // of the clamped gate (PL_ACT_CLAMPED)
    int plain;             // an expert is down(act(up x)): w_gu holds up rows alone, [E, F, W]
    // An expert of another size that every row of a router's choice names last, as number `shared_at` (-1: there is none).
    int shared_at, shared_F;
    const void* shared_gu; // [2 shared_F, W], or [shared_F, W] where plain
    const void* shared_down;  // [W, shared_F]
};

// The values of a row's pairs lie one behind the other in h: pair c from c F on, the shared expert's, the last, of another length.
__host__ __device__ static inline int moe_row_values(const MoeArgs& a) {
    return a.shared_at >= 0 ? (a.top - 1) * a.F + a.shared_F : a.top * a.F;
}

// The expert of pair (t, c), or -1: the router's choice, or the table's row of the token's id.
__device__ __forceinline__ int moe_pair_expert(const MoeArgs& a, int t, int c) {
    if (a.choice != nullptr) return a.choice[static_cast<size_t>(t) * a.top + c];
    const int id = moe_token(a.ids, a.src, a.fed, t);
    if (id < 0 || id >= a.vocab) return -1;
    return a.table[static_cast<size_t>(id) * a.top + c];
}

// The outputs of a step's pairs, to be added up a row: row t is the sum over c of weight[t * top + c] * y[slot of (t, c)], the
// choices in their order.  The slot is slot_of[t * top + c] or, where slot_of is null, t * top + c itself; a pair without one (negative,
// or, without slot_of, without an expert) adds nothing.  y may come in `splits` copies, `split_stride` floats apart, each a
// stretch of the product's inner width: a pair's copies are added in their order.
struct ExpertSum {
    const float* y;        // [slots, W]; null: nothing to add
    const int* slot_of;
    const int* choice;     // [n, top] or null
    const float* weight;   // [n, top]; null: every pair counts 1 / top
    int top, splits;
    size_t split_stride;
};

__device__ __forceinline__ int expert_slot(const ExpertSum& s, int t, int c) {
    const int p = t * s.top + c;
    if (s.slot_of != nullptr) return s.slot_of[p];
    return s.choice != nullptr && s.choice[p] < 0 ? -1 : p;
}

__device__ __forceinline__ float4 expert_output(const ExpertSum& s, int slot, int W, int w) {
    float4 v = *reinterpret_cast<const float4*>(s.y + static_cast<size_t>(slot) * W + w);
    for (int k = 1; k < s.splits; ++k) {
        const float4 more = *reinterpret_cast<const float4*>(s.y + k * s.split_stride + static_cast<size_t>(slot) * W + w);
        v.x += more.x;
        v.y += more.y;
        v.z += more.z;
        v.w += more.w;
    }
    return v;
}
