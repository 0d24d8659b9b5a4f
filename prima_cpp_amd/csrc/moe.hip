// moe.hip — routing of a step's tokens to experts. Up to 64 tokens: one workgroup scores, selects and sorts (expert by expert, tokens in order). More: a wave per token
// selects and takes a place in its expert's list, then every workgroup sorts its share of the pairs (the order inside an expert does not enter any sum).
#include "pm355_route.h"
#include "pm355_kernels.h"

namespace {

// exclusive prefix of the experts' counts in LDS: off[0 .. E]; one wave
__device__ __forceinline__ void prefix(const int * count, int E, int * off) {
    const int lane = threadIdx.x & 63;
    int carry = 0;
    for (int e0 = 0; e0 < E; e0 += 64) {
        const int v = e0 + lane < E ? count[e0 + lane] : 0;
        int s = v;
        for (int o = 1; o < 64; o *= 2) { const int u = __shfl_up(s, o); if (lane >= o) s += u; }
        if (e0 + lane < E) off[e0 + lane] = carry + s - v;
        carry += __shfl(s, 63);
    }
    if (lane == 0) off[E] = carry;
}
// which experts have pairs, and their tiles; one wave
__device__ __forceinline__ void lists(const int * off, const pm_route & r, int want_tiles) {
    const int lane = threadIdx.x & 63;
    int n_act = 0, n_tile = 0;
    for (int e0 = 0; e0 < r.E; e0 += 64) {
        const int e = e0 + lane, n = e < r.E ? off[e + 1] - off[e] : 0;
        const uint64_t on = __builtin_amdgcn_ballot_w64(n > 0);
        if (n > 0) r.active[1 + n_act + __popcll(on & ((1ull << lane) - 1))] = e;
        n_act += __popcll(on);
        if (!want_tiles) continue;
        const int tiles = (n + r.tile - 1) / r.tile;
        int s = tiles;
        for (int o = 1; o < 64; o *= 2) { const int u = __shfl_up(s, o); if (lane >= o) s += u; }
        for (int i = 0; i < tiles; ++i) {
            int32_t * t = r.tiles + 1 + 3 * (n_tile + s - tiles + i);
            t[0] = e; t[1] = off[e] + i * r.tile; t[2] = n - i * r.tile < r.tile ? n - i * r.tile : r.tile;
        }
        n_tile += __shfl(s, 63);
    }
    if (lane == 0) { r.active[0] = n_act; if (want_tiles) r.tiles[0] = n_tile; }
}

// T <= 64 tokens. LDS: [16 waves][E] scores, [16][groups], count[E], off[E + 1], ids [T * top]
__global__ __launch_bounds__(1024) void route_one_kernel(pm_route r, int T, int want_tiles) {
    extern __shared__ __attribute__((aligned(16))) float sm[];
    const int wave = threadIdx.x >> 6, lane = threadIdx.x & 63, pairs = T * r.top;
    float * s = sm + wave * r.E, * gs = sm + 16 * r.E + wave * r.groups;
    int * off = (int *) (sm + 16 * (r.E + r.groups)), * count = off + r.E + 1, * ids = count + r.E;
    float * ws = (float *) (ids + pairs);
    for (int t = wave; t < T; t += 16) {
        route_token(r.logits + (size_t) t * r.ldl, r.E, r.top, r.groups, r.keep, s, gs, ids + t * r.top, ws + t * r.top);
        for (int k = lane; k < r.top; k += 64) { r.id[t * r.top + k] = ids[t * r.top + k]; r.w[t * r.top + k] = ws[t * r.top + k]; }
    }
    __syncthreads();
    for (int e = threadIdx.x; e < r.E; e += 1024) {
        int n = 0;
        for (int i = 0; i < pairs; ++i) n += ids[i] == e;
        count[e] = n;
    }
    __syncthreads();
    if (wave == 0) prefix(count, r.E, off);
    __syncthreads();
    if (wave == 0) lists(off, r, want_tiles);
    for (int e = threadIdx.x; e <= r.E; e += 1024) {
        int at = off[e];
        r.off[e] = at;
        if (e < r.E && count[e]) for (int i = 0; i < pairs; ++i) if (ids[i] == e) r.order[at++] = i;
    }
}

// 32 tokens per workgroup: places among its own pairs by LDS counters, then one global counter update per expert
constexpr int SEL_TOK = 32;
__global__ __launch_bounds__(1024) void route_select_kernel(pm_route r, int T) {
    extern __shared__ __attribute__((aligned(16))) float sm[];
    const int wave = threadIdx.x >> 6, t0 = blockIdx.x * SEL_TOK, n = (T - t0 < SEL_TOK ? T - t0 : SEL_TOK) * r.top;
    int * count = (int *) sm, * ids = count + r.E;
    float * w = (float *) (ids + SEL_TOK * r.top), * s = w + SEL_TOK * r.top + wave * (r.E + r.groups);
    for (int e = threadIdx.x; e < r.E; e += 1024) count[e] = 0;
    for (int i = wave; i < SEL_TOK && t0 + i < T; i += 16)
        route_token(r.logits + (size_t) (t0 + i) * r.ldl, r.E, r.top, r.groups, r.keep, s, s + r.E, ids + i * r.top, w + i * r.top);
    __syncthreads();
    for (int i = threadIdx.x; i < n; i += 1024) {
        r.id[t0 * r.top + i] = ids[i]; r.w[t0 * r.top + i] = w[i];
        ((int *) w)[i] = atomicAdd(count + ids[i], 1);     // (the weight has been stored: its place takes over)
    }
    __syncthreads();
    for (int e = threadIdx.x; e < r.E; e += 1024) if (count[e]) count[e] = atomicAdd(r.count + e, count[e]);
    __syncthreads();
    for (int i = threadIdx.x; i < n; i += 1024) r.pos[t0 * r.top + i] = count[ids[i]] + ((int *) w)[i];
}
__global__ __launch_bounds__(256) void route_place_kernel(pm_route r, int pairs, int want_tiles) {
    extern __shared__ __attribute__((aligned(16))) int cnt[];
    int * off = cnt + r.E;
    for (int e = threadIdx.x; e < r.E; e += 256) cnt[e] = r.count[e];
    __syncthreads();
    if (threadIdx.x < 64) prefix(cnt, r.E, off);
    __syncthreads();
    if (blockIdx.x == 0) {
        if (threadIdx.x < 64) lists(off, r, want_tiles);
        for (int e = threadIdx.x; e <= r.E; e += 256) r.off[e] = off[e];
    }
    const int p = blockIdx.x * 256 + threadIdx.x;
    if (p < pairs) r.order[off[r.id[p]] + r.pos[p]] = p;
}

} // namespace

void pm_launch_route(const pm_route & r, int T, int want_tiles, hipStream_t st) {
    const int pairs = T * r.top;
    if (T <= PM_ROUTE_ONE_MAX) {
        const size_t lds = (size_t) 16 * (r.E + r.groups) * 4 + (size_t) (2 * r.E + 1 + 2 * pairs) * 4;
        pm_allow_big_lds((const void *) route_one_kernel, lds);
        if (lds <= 150 * 1024) { hipLaunchKernelGGL(route_one_kernel, dim3(1), dim3(1024), lds, st, r, T, want_tiles); return; }
    }
    const size_t lds = ((size_t) r.E + 2 * SEL_TOK * r.top + 16 * (r.E + r.groups)) * 4;      // (at most 150 KB: E, groups <= 1024, top <= 64)
    pm_allow_big_lds((const void *) route_select_kernel, lds);
    hipLaunchKernelGGL(route_select_kernel, dim3((T + SEL_TOK - 1) / SEL_TOK), dim3(1024), lds, st, r, T);
    hipLaunchKernelGGL(route_place_kernel, dim3((pairs + 255) / 256), dim3(256), (size_t) (2 * r.E + 1) * 4, st, r, pairs, want_tiles);
}
