// route.h -- one row's choice of experts by one wave (kernels_moe.hip, kernels_residual.hip).
#pragma once
#include "common.h"
#include "decoder.h"

namespace pgmi {

// LDS written by some lanes of a wave and read by others (a wave's LDS operations complete in order)
__device__ __forceinline__ void wave_sync() {
    __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront");
    __builtin_amdgcn_wave_barrier();
}

// floats in the order of their values, as unsigned integers: a total order, whatever the bits are
__device__ __forceinline__ uint32_t order_key(float f) {
    const uint32_t b = __float_as_uint(f);
    return b & 0x80000000u ? ~b : b | 0x80000000u;
}

// LDS words of one row: scores, choice keys (padded to 4), group keys
__host__ __device__ inline int route_words(int n, int groups) { return 2 * ((n + 3) & ~3) + ((groups + 3) & ~3); }

// sc[0 .. n) holds the row's logits and receives their softmax; choice = score + correction(expert).  A group's key is its largest
// choice; experts outside the `keep` best groups cannot be chosen.  The place of an expert is the number of those before
// it (larger choice, or equal and a smaller index), so exactly `top` places 0 .. top-1 are taken, each by one lane:
// take(place, expert, score).
template <typename C, typename F>
__device__ __forceinline__ void route_row(float* sc, C correction, int n, int groups, int keep, int top, int lane, F take) {
    const int np = (n + 3) & ~3, gs = n / groups;
    uint32_t* key = reinterpret_cast<uint32_t*>(sc + np);
    uint32_t* gr = key + np;
    const bool limited = keep < groups;
    float mx = -INFINITY, sum = 0.0f;
    for (int c = lane; c < n; c += 64) mx = fmaxf(mx, sc[c]);
    mx = wave_max(mx);
    for (int c = lane; c < n; c += 64) {
        const float e = expf(sc[c] - mx);
        sc[c] = e;
        sum += e;
    }
    const float inv = 1.0f / wave_sum(sum);
    if (limited)
        for (int g = lane; g < groups; g += 64) gr[g] = 0;
    wave_sync();
    for (int c = lane; c < np; c += 64) {
        uint32_t k = 0;  // pads: after every expert
        if (c < n) {
            const float s = sc[c] * inv;
            sc[c] = s;
            k = order_key(s + correction(c));
            if (limited) atomicMax(&gr[c / gs], k);
        }
        key[c] = k;
    }
    wave_sync();
    if (limited) {
        for (int c = lane; c < n; c += 64) {
            const int g = c / gs;
            const uint32_t k = gr[g];
            int before = 0;
            for (int q = 0; q < groups; ++q) before += gr[q] > k || (gr[q] == k && q < g);
            if (before >= keep) key[c] = 0;
        }
        wave_sync();
    }
    for (int c = lane; c < n; c += 64) {
        const uint32_t k = key[c];
        int before = 0;
#pragma unroll 4
        for (int j = 0; j < np; j += 4) {
            const uint4 q = *reinterpret_cast<const uint4*>(key + j);
            before += q.x > k || (q.x == k && j < c);
            before += q.y > k || (q.y == k && j + 1 < c);
            before += q.z > k || (q.z == k && j + 2 < c);
            before += q.w > k || (q.w == k && j + 3 < c);
        }
        if (before < top) take(before, c, sc[c]);
    }
}

}  // namespace pgmi
