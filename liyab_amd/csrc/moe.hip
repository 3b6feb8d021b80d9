// Routing of a mixture of experts: who goes where, before the experts' products run
// (grouped_product.hip).
//
// liyab_moe_route: from each token's 32-bit router logits the `top` experts with the largest
// logits (among equal logits the lower number first) and their weights, the softmax over the chosen
// logits alone, in 32-bit. ids and weights [n, top]: entry t * top + k is token t's k-th choice.
// mode 1: the choice among groups of experts instead (route_token_groups): softmax over all experts, the best
// groups only, weights divided by their sum.
// mode 2: scores s = 1 / (1 + exp(-z)), the choice by c = s + correction (route_wave): a group's score is the sum of its two
// largest c, only experts of the best groups, of those the `top` largest c; weights are the chosen s as they are. A wave routes a
// token (its scores in LDS, an expert a lane), since every score costs an exponential.
// mode 3: as mode 2 with scores s = softmax(z) over all outputs; weights are scale * s of the chosen ones.
// Modes 2 and 3: outputs from `n_listed` on are identity experts, whose result is the token's own input: they get the id -1, so that no
// list holds them, and whoever adds a token's rows up puts the input there. With `extra`, a token has one more entry behind its `top`: expert
// n_listed, which every token takes, weighted sigmoid(z[E]) (a logit of its own behind the router's).
//
// liyab_moe_align: the entries listed by expert, each expert's stretch padded to whole tiles of
// `block` places: rows_list [max_tiles * block] (an entry's number, -1 for an empty place) and
// tile_group [max_tiles] (the expert of each tile, -1 for a tile that is not used). max_tiles is
// a bound that the step's sizes fix (entries / block + min(experts, entries), rounded up), so
// that the products' grids do not depend on where the tokens went. One workgroup.
//
// liyab_moe_route_align: both in one launch, for steps of at most 1,024 tokens (modes 2 and 3: kWaveRouteTokens).
#include "common.h"
#include "launchers.h"

namespace liyab {

constexpr int kMaxTop = 64;

// One token's choice: the `top` largest of its E logits (the lower number among equals) and the softmax over them.
__device__ __forceinline__ void route_token(const float* __restrict__ z, int E, int top, int* __restrict__ ids, float* __restrict__ weights) {
    int chosen[kMaxTop];
    float value[kMaxTop];
    for (int k = 0; k < top; ++k) {
        int best = -1;
        float bv = 0.0f;
        for (int e = 0; e < E; ++e) {
            bool taken = false;
            for (int j = 0; j < k; ++j) taken = taken || chosen[j] == e;
            const float v = z[e];
            if (!taken && (best < 0 || v > bv)) {
                best = e;
                bv = v;
            }
        }
        chosen[k] = best;
        value[k] = bv;
    }
    float sum = 0.0f;
    const float largest = value[0];  // the first choice holds the largest logit
    for (int k = 0; k < top; ++k) {
        value[k] = expf(value[k] - largest);
        sum += value[k];
    }
    for (int k = 0; k < top; ++k) {
        ids[k] = chosen[k];
        weights[k] = value[k] / sum;
    }
}

// One token's choice among groups of experts: s = softmax(z) over all experts; the experts form `n_groups` equal groups of
// neighbours, a group's score is its largest s, and only experts of the `keep` best groups (the lower number among equals)
// can be chosen; of those the `top` largest s (the lower number among equals), weighted s / (their sum + 1e-20).
constexpr int kMaxGroups = 64;
constexpr float kWeightFloor = 1e-20f;

__device__ __forceinline__ void route_token_groups(const float* __restrict__ z, int E, int top, int n_groups, int keep, int* __restrict__ ids,
                                                   float* __restrict__ weights) {
    float largest = z[0];
    for (int e = 1; e < E; ++e) largest = fmaxf(largest, z[e]);
    float total = 0.0f;
    for (int e = 0; e < E; ++e) total += expf(z[e] - largest);
    const int per = E / n_groups;
    uint64_t kept = 0;  // the groups whose experts can be chosen
    for (int k = 0; k < keep; ++k) {
        int best = -1;
        float bv = 0.0f;
        for (int g = 0; g < n_groups; ++g) {
            if ((kept >> g) & 1) continue;
            float gv = z[g * per];
            for (int e = 1; e < per; ++e) gv = fmaxf(gv, z[g * per + e]);  // (the largest score is the largest logit's)
            if (best < 0 || gv > bv) {
                best = g;
                bv = gv;
            }
        }
        kept |= uint64_t(1) << best;
    }
    int chosen[kMaxTop];
    float value[kMaxTop];
    float sum = 0.0f;
    for (int k = 0; k < top; ++k) {
        int best = -1;
        float bv = 0.0f;
        for (int e = 0; e < E; ++e) {
            if (!((kept >> (e / per)) & 1)) continue;
            bool taken = false;
            for (int j = 0; j < k; ++j) taken = taken || chosen[j] == e;
            const float v = z[e];
            if (!taken && (best < 0 || v > bv)) {
                best = e;
                bv = v;
            }
        }
        chosen[k] = best;
        value[k] = expf(bv - largest) / total;
        sum += value[k];
    }
    for (int k = 0; k < top; ++k) {
        ids[k] = chosen[k];
        weights[k] = value[k] / (sum + kWeightFloor);
    }
}

// One token's choice by a wave, c (LDS, E floats) its own: see mode 2 above. Among equals the lower number first; an expert that
// cannot be chosen, or has been, is minus infinity (c itself can be negative).
constexpr int kMaxWaveExperts = 2048;
constexpr int kWaveRouteTokens = 64;  // tokens a launch of one workgroup routes at most (sixteen waves, four each)

// What a wave's lanes wrote to LDS is there for its other lanes.
__device__ __forceinline__ void wave_lds_order() { asm volatile("s_waitcnt lgkmcnt(0)" ::: "memory"); }

struct RouteArgs {
    int mode, n_groups, keep;
    const float* correction;
    float scale;          // mode 3: on the weights
    int n_listed, extra;  // modes 2 and 3: see the head of this file
};

__device__ __forceinline__ void route_wave(const float* __restrict__ z, const RouteArgs& ra, int E, int top, int* __restrict__ ids, float* __restrict__ weights,
                                           float* c) {
    const int lane = threadIdx.x % kWave, n_groups = ra.n_groups, keep = ra.keep;
    const float* correction = ra.correction;
    float largest = 0.0f, norm = 1.0f;  // mode 3: a score is exp(z - largest) * norm
    if (ra.mode == 3) {
        largest = -INFINITY;
        for (int e = lane; e < E; e += kWave) largest = fmaxf(largest, z[e]);
        largest = wave_max(largest);
        float total = 0.0f;
        for (int e = lane; e < E; e += kWave) total += expf(z[e] - largest);
        norm = 1.0f / wave_sum(total);
    }
    auto score = [&](int e) { return ra.mode == 3 ? expf(z[e] - largest) * norm : 1.0f / (1.0f + expf(-z[e])); };
    for (int e = lane; e < E; e += kWave) c[e] = score(e) + (correction != nullptr ? correction[e] : 0.0f);
    wave_lds_order();
    const int per = E / n_groups;
    uint64_t kept = ~uint64_t(0);
    if (keep < n_groups) {
        kept = 0;
        float score = -INFINITY;  // lane g: group g's
        if (lane < n_groups) {
            float a = -INFINITY, b = -INFINITY;  // its two largest
            for (int e = 0; e < per; ++e) {
                const float v = c[lane * per + e];
                b = fmaxf(b, fminf(a, v));
                a = fmaxf(a, v);
            }
            score = per > 1 ? a + b : a;
        }
        for (int k = 0; k < keep; ++k) {
            float bv = score;
            int bi = lane < n_groups ? lane : kMaxGroups + lane;
            wave_argmax(bv, bi);
            kept |= uint64_t(1) << (bi % kMaxGroups);
            if (lane == bi) score = -INFINITY;
        }
    }
    for (int k = 0; k < top; ++k) {
        float bv = -INFINITY;
        int bi = E;
        for (int e = lane; e < E; e += kWave) {
            const float v = ((kept >> (e / per)) & 1) || n_groups == 1 ? c[e] : -INFINITY;
            if (v > bv) {
                bv = v;
                bi = e;
            }
        }
        wave_argmax(bv, bi);
        const int best = min(bi, E - 1);
        if (lane == 0) {
            ids[k] = best < ra.n_listed ? best : -1;
            weights[k] = score(best) * ra.scale;
        }
        if (lane == best % kWave) c[best] = -INFINITY;
        wave_lds_order();
    }
    if (ra.extra && lane == 0) {
        ids[top] = ra.n_listed;
        weights[top] = 1.0f / (1.0f + expf(-z[E]));
    }
}

// The same for one group of at most 64 outputs: an output a lane, its score in a register; zl is the lane's logit, and with `extra` lane 0 knows the
// token's own one. No trip through LDS.
__device__ __forceinline__ void route_wave_lane(float zl, float own, const RouteArgs& ra, int E, int top, int* __restrict__ ids, float* __restrict__ weights) {
    const int lane = threadIdx.x % kWave;
    const bool real = lane < E;
    float s;
    if (ra.mode == 3) {
        const float v = real ? expf(zl - wave_max(real ? zl : -INFINITY)) : 0.0f;
        s = v * (1.0f / wave_sum(v));
    } else {
        s = 1.0f / (1.0f + expf(-zl));
    }
    float c = real ? s + (ra.correction != nullptr ? ra.correction[lane] : 0.0f) : -INFINITY;
    for (int k = 0; k < top; ++k) {
        float bv = c;
        int bi = real ? lane : kWave + lane;
        wave_argmax(bv, bi);
        const int best = min(bi, E - 1);
        if (lane == best) {
            ids[k] = best < ra.n_listed ? best : -1;
            weights[k] = s * ra.scale;
            c = -INFINITY;
        }
    }
    if (ra.extra && lane == 0) {
        ids[top] = ra.n_listed;
        weights[top] = 1.0f / (1.0f + expf(-own));
    }
}
__device__ __forceinline__ bool routes_in_lanes(const RouteArgs& ra, int E) { return E <= kWave && ra.keep == ra.n_groups; }

// a wave a token, four waves a workgroup
__global__ void __launch_bounds__(256)
moe_route_wave_kernel(const float* __restrict__ logits, int64_t ld, RouteArgs ra, int n, int E, int top, int* __restrict__ ids, float* __restrict__ weights) {
    extern __shared__ int sh[];
    const int wave = threadIdx.x / kWave, t = blockIdx.x * 4 + wave;
    if (t >= n) return;
    const int64_t at = static_cast<int64_t>(t) * (top + ra.extra);
    if (routes_in_lanes(ra, E)) {
        const float* z = logits + static_cast<int64_t>(t) * ld;
        route_wave_lane(z[min(static_cast<int>(threadIdx.x) % kWave, E - 1)], z[ra.extra ? E : 0], ra, E, top, ids + at, weights + at);
        return;
    }
    route_wave(logits + static_cast<int64_t>(t) * ld, ra, E, top, ids + at, weights + at, reinterpret_cast<float*>(sh) + wave * E);
}

// mode 0: the largest logits, softmax over the chosen ones; mode 1: softmax over all, groups, weights by their sum
__device__ __forceinline__ void route_any(const float* __restrict__ z, int E, int top, int mode, int n_groups, int keep, int* __restrict__ ids,
                                          float* __restrict__ weights) {
    if (mode == 1) route_token_groups(z, E, top, n_groups, keep, ids, weights);
    else route_token(z, E, top, ids, weights);
}

__global__ void __launch_bounds__(256)
moe_route_kernel(const float* __restrict__ logits, int64_t ld, int n, int E, int top, int* __restrict__ ids, float* __restrict__ weights,
                 int mode, int n_groups, int keep) {
    const int t = blockIdx.x * 256 + threadIdx.x;
    if (t >= n) return;
    route_any(logits + static_cast<int64_t>(t) * ld, E, top, mode, n_groups, keep, ids + static_cast<int64_t>(t) * top, weights + static_cast<int64_t>(t) * top);
}

// The entries of `ids` listed by expert in tiles of `block` places; one workgroup of 1,024 threads runs this.
__device__ __forceinline__ void align_entries(const int* __restrict__ ids, int n_entries, int E, int block, int* __restrict__ rows_list,
                                              int* __restrict__ tile_group, int max_tiles, int* sh) {
    int* counts = sh;     // [E]
    int* first = sh + E;  // [E + 1]: the first place of each expert
    const int tid = threadIdx.x;
    for (int e = tid; e < E; e += 1024) counts[e] = 0;
    for (int i = tid; i < max_tiles * block; i += 1024) rows_list[i] = -1;
    for (int i = tid; i < max_tiles; i += 1024) tile_group[i] = -1;
    __syncthreads();
    for (int i = tid; i < n_entries; i += 1024) {
        const int e = ids[i];
        if (e >= 0 && e < E) atomicAdd(&counts[e], 1);
    }
    __syncthreads();
    if (tid == 0) {
        int at = 0;
        for (int e = 0; e < E; ++e) {
            first[e] = at;
            const int tiles = (counts[e] + block - 1) / block;
            for (int i = 0; i < tiles; ++i)
                if (at / block + i < max_tiles) tile_group[at / block + i] = e;
            at += tiles * block;
            counts[e] = 0;  // counts the entries placed so far from here on
        }
        first[E] = at;
    }
    __syncthreads();
    for (int i = tid; i < n_entries; i += 1024) {
        const int e = ids[i];
        if (e < 0 || e >= E) continue;
        const int place = first[e] + atomicAdd(&counts[e], 1);
        if (place < max_tiles * block) rows_list[place] = i;
    }
}

__global__ void __launch_bounds__(1024)
moe_align_kernel(const int* __restrict__ ids, int n_entries, int E, int block, int* __restrict__ rows_list, int* __restrict__ tile_group,
                 int max_tiles) {
    extern __shared__ int sh[];
    align_entries(ids, n_entries, E, block, rows_list, tile_group, max_tiles, sh);
}

// Both in one launch for steps of at most 1,024 tokens: a thread routes a token, then the workgroup lists the entries.
__global__ void __launch_bounds__(1024)
moe_route_align_kernel(const float* __restrict__ logits, int64_t ld, int n, int E, int top, int* __restrict__ ids, float* __restrict__ weights,
                       int block, int* __restrict__ rows_list, int* __restrict__ tile_group, int max_tiles, RouteArgs ra) {
    extern __shared__ int sh[];
    const int t = threadIdx.x;
    if (ra.mode >= 2) {  // a wave a token, sixteen at a time
        const int wave = t / kWave;
        if (routes_in_lanes(ra, E)) {
            constexpr int kEach = kWaveRouteTokens / (1024 / kWave);  // tokens a wave: all their logits are asked for together
            float zl[kEach], own[kEach];
#pragma unroll
            for (int j = 0; j < kEach; ++j) {
                const float* z = logits + static_cast<int64_t>(min(wave + j * (1024 / kWave), n - 1)) * ld;
                zl[j] = z[min(t % kWave, E - 1)];
                own[j] = z[ra.extra ? E : 0];
            }
#pragma unroll
            for (int j = 0; j < kEach; ++j) {
                const int i = wave + j * (1024 / kWave);
                const int64_t at = static_cast<int64_t>(i) * (top + ra.extra);
                if (i < n) route_wave_lane(zl[j], own[j], ra, E, top, ids + at, weights + at);
            }
        } else for (int i = wave; i < n; i += 1024 / kWave) {
            const int64_t at = static_cast<int64_t>(i) * (top + ra.extra);
            route_wave(logits + static_cast<int64_t>(i) * ld, ra, E, top, ids + at, weights + at, reinterpret_cast<float*>(sh) + wave * E);
        }
    } else if (t < n) route_any(logits + static_cast<int64_t>(t) * ld, E, top, ra.mode, ra.n_groups, ra.keep, ids + static_cast<int64_t>(t) * top, weights + static_cast<int64_t>(t) * top);
    __syncthreads();  // (the ids are read back by other threads of this workgroup)
    align_entries(ids, n * (top + ra.extra), ra.n_listed + ra.extra, block, rows_list, tile_group, max_tiles, sh);
}

}  // namespace liyab

using namespace liyab;

// ids and weights: [n, top + extra]. n_listed, extra: see the head of this file (n_experts and 0 outside modes 2 and 3).
extern "C" int liyab_moe_route(const float* logits, int64_t ld, int n, int n_experts, int top, int* ids, float* weights, int mode, int n_groups,
                               int keep, const float* correction, float scale, int n_listed, int extra, hipStream_t stream) {
    LIYAB_REQUIRE(logits && ids && weights, "moe_route: null pointer");
    LIYAB_REQUIRE(mode == 0 || (mode >= 1 && mode <= 3 && n_groups >= 1 && n_groups <= kMaxGroups && n_experts % n_groups == 0 && keep >= 1 && keep <= n_groups &&
                                top <= keep * (n_experts / n_groups)),
                  "moe_route: %d of %d groups of %d experts do not hold %d choices (at most %d groups)", keep, n_groups, n_experts, top, kMaxGroups);
    LIYAB_REQUIRE(n >= 0 && n_experts > 0 && top >= 1 && top <= n_experts && top <= kMaxTop && ld >= n_experts,
                  "moe_route: bad sizes n=%d experts=%d top=%d (at most %d choices a token)", n, n_experts, top, kMaxTop);
    LIYAB_REQUIRE(mode < 2 || n_experts <= kMaxWaveExperts, "moe_route: %d experts; at most %d are taken in this mode", n_experts, kMaxWaveExperts);
    LIYAB_REQUIRE(n_listed >= 1 && n_listed <= n_experts && (extra == 0 || extra == 1) && (mode >= 2 || (n_listed == n_experts && extra == 0)) && ld >= n_experts + extra,
                  "moe_route: %d listed of %d outputs, %d entries for every token do not go with this mode", n_listed, n_experts, extra);
    if (n == 0) return 0;
    if (mode >= 2) {
        const RouteArgs ra{mode, n_groups, keep, correction, scale, n_listed, extra};
        moe_route_wave_kernel<<<(n + 3) / 4, 256, 4 * n_experts * sizeof(float), stream>>>(logits, ld, ra, n, n_experts, top, ids, weights);
        return check_launch("moe_route");
    }
    moe_route_kernel<<<(n + 255) / 256, 256, 0, stream>>>(logits, ld, n, n_experts, top, ids, weights, mode, n_groups, keep);
    return check_launch("moe_route");
}

extern "C" int liyab_moe_align(const int* ids, int n_entries, int n_experts, int block, int* rows_list, int* tile_group, int max_tiles,
                               hipStream_t stream) {
    LIYAB_REQUIRE(ids && rows_list && tile_group, "moe_align: null pointer");
    LIYAB_REQUIRE(n_entries >= 0 && n_experts > 0 && n_experts <= 4096 && block > 0, "moe_align: bad sizes (at most 4,096 experts)");
    LIYAB_REQUIRE(static_cast<int64_t>(max_tiles) * block >= static_cast<int64_t>(n_entries) + static_cast<int64_t>(n_entries < n_experts ? n_entries : n_experts) * (block - 1),
                  "moe_align: %d tiles of %d places do not hold %d entries of %d experts", max_tiles, block, n_entries, n_experts);
    if (n_entries == 0) return 0;
    moe_align_kernel<<<1, 1024, (2 * n_experts + 1) * sizeof(int), stream>>>(ids, n_entries, n_experts, block, rows_list, tile_group, max_tiles);
    return check_launch("moe_align");
}

extern "C" int liyab_moe_route_align(const float* logits, int64_t ld, int n, int n_experts, int top, int* ids, float* weights, int block,
                                     int* rows_list, int* tile_group, int max_tiles, int mode, int n_groups, int keep, const float* correction,
                                     float scale, int n_listed, int extra, hipStream_t stream) {
    LIYAB_REQUIRE(n <= 1024, "moe_route_align: %d tokens; one workgroup routes at most 1,024 (moe_route and moe_align take more)", n);
    if (const int rc = liyab_moe_route(logits, ld, 0, n_experts, top, ids, weights, mode, n_groups, keep, correction, scale, n_listed, extra, stream)) return rc;  // (the checks of both,
    const int listed = n_listed + extra;
    if (const int rc = liyab_moe_align(ids, 0, listed, block, rows_list, tile_group, max_tiles, stream)) return rc;    //  nothing launched)
    LIYAB_REQUIRE(n >= 0 && static_cast<int64_t>(max_tiles) * block >= static_cast<int64_t>(n) * (top + extra) + static_cast<int64_t>(n * (top + extra) < listed ? n * (top + extra) : listed) * (block - 1),
                  "moe_route_align: %d tiles of %d places do not hold %d entries of %d experts", max_tiles, block, n * (top + extra), listed);
    LIYAB_REQUIRE(mode < 2 || (n <= kWaveRouteTokens && n_experts <= 512), "moe_route_align: %d tokens of %d experts; modes 2 and 3 take %d of 512 here", n, n_experts, kWaveRouteTokens);
    if (n == 0) return 0;
    const size_t smem = sizeof(int) * (mode >= 2 ? (1024 / kWave) * static_cast<size_t>(n_experts) + 4 : 2 * static_cast<size_t>(n_experts) + 1);  // (the scores; then the lists' counts)
    const RouteArgs ra{mode, n_groups, keep, correction, scale, n_listed, extra};
    moe_route_align_kernel<<<1, 1024, smem, stream>>>(logits, ld, n, n_experts, top, ids, weights, block, rows_list, tile_group, max_tiles, ra);
    return check_launch("moe_route_align");
}
