// pm355_route.h — routing of one token to its experts by one wave (moe.hip, and the prologue of the few-token expert products in dense_small.hip).
#pragma once
#include "pm355_dense.h"

#ifdef __HIPCC__
// LDS of one routing wave: s [E] scores, gs [groups]. ids / w receive `top` entries, largest score first (equal scores: lower index first). E <= 1024, groups <= 1024.
// Ranks instead of repeated maxima: every lane counts, for its own experts, how many stand in front of them.
__device__ __forceinline__ void wave_fence() { __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "wavefront"); __builtin_amdgcn_wave_barrier(); }
__device__ __forceinline__ void route_token(const float * z, int E, int top, int groups, int keep, float * s, float * gs, int * ids, float * w) {
    const int lane = threadIdx.x & 63;
    float mx = -INFINITY, sum = 0.0f;
    for (int k = lane; k < top; k += 64) { ids[k] = 0; w[k] = 0.0f; }        // (a row of NaNs has no ranks)
    for (int e = lane; e < E; e += 64) { const float v = ld_g(z + e); s[e] = v; mx = fmaxf(mx, v); }
    mx = wave_max(mx);
    for (int e = lane; e < E; e += 64) { const float v = expf(s[e] - mx); s[e] = v; sum += v; }
    sum = wave_sum(sum);
    for (int e = lane; e < E; e += 64) s[e] /= sum;
    wave_fence();
    if (keep < groups) {
        const int per = E / groups;
        for (int g = lane; g < groups; g += 64) {
            float m = s[g * per];
            for (int i = 1; i < per; ++i) m = fmaxf(m, s[g * per + i]);
            gs[g] = m;
        }
        wave_fence();
        for (int e = lane; e < E; e += 64) {
            const int g = e / per;
            const float m = gs[g];
            int front = 0;
            for (int i = 0; i < groups; ++i) { const float o = gs[i]; front += o > m || (o == m && i < g); }
            if (front >= keep) s[e] = -1.0f;               // (only this lane reads s[e] before the fence)
        }
        wave_fence();
    }
    for (int e = lane; e < E; e += 64) {
        const float m = s[e];
        int front = 0;
        for (int i = 0; i < E; ++i) { const float o = s[i]; front += o > m || (o == m && i < e); }
        if (front < top) { ids[front] = e; w[front] = fmaxf(m, 0.0f); }
    }
    wave_fence();
}
#endif
