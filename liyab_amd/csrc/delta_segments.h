// What recurrences of the delta-rule kind share when a long portion runs in segments side by side: a head's state S [D, V] of a
// request moves by S_t = A_t S_(t-1) + (an outer product), A_t a D x D matrix, so a segment's end is P S_start + Z with P the product
// of its A_t and Z its end from a zero state.
#pragma once

#include "common.h"

namespace liyab {

constexpr int kDeltaCols = 16;    // columns of S a wave
constexpr int kDeltaSplit = 4;    // lanes that share a column's rows
constexpr int kDeltaWaves = 4;    // waves a workgroup, each with work of its own

struct DeltaSegments {
    const float* state;       // the heads' matrices [H, D, V] of slot 0; a slot is state_stride floats further
    int64_t state_stride;
    int n_slots;
    const int* seq_starts;
    const int* positions;
    const int* state_slots;
    int n_seqs, H, D, V;
    int seg_tokens;
};

// segment `g` of the step in the order of the requests: its request and rows; false past the last segment
__device__ __forceinline__ bool find_segment(const int* seq_starts, int n_seqs, int seg_tokens, int g, int& s, int& begin, int& end, bool& last) {
    for (s = 0; s < n_seqs; ++s) {
        const int b = seq_starts[s], len = seq_starts[s + 1] - b;
        const int n_seg = (len + seg_tokens - 1) / seg_tokens;
        if (g < n_seg) {
            begin = b + g * seg_tokens;
            end = min(begin + seg_tokens, b + len);
            last = g == n_seg - 1;
            return true;
        }
        g -= n_seg;
    }
    return false;
}

// Between the two passes over the segments: the state each segment starts from. A workgroup a (request, head, block of 16
// columns) walks the request's segments in order, S <- P S + Z, and leaves in seg_start what each segment starts from (the
// first: the slot's state, or zeros at position 0); an array of its own, named as such to the compiler, so that no load of a
// later segment's Z or P has to wait behind a store. A thread holds rows ib, ib + 16, ... of one column; the columns' block
// of S lies in LDS; P goes through LDS in tiles of 64 x 64, the next tile fetched into registers while this one is used.
constexpr int kCombTile = 64, kCombStride = kCombTile + 4;  // (rows 68 floats apart: four rows read together fall into different banks)
constexpr int kCombMaxD = 256;

static __global__ void __launch_bounds__(256)
delta_combine_kernel(DeltaSegments a, const float* __restrict__ seg_z, const float* __restrict__ seg_p, float* __restrict__ seg_start) {
    __shared__ __attribute__((aligned(16))) float Pt[kCombTile * kCombStride];
    __shared__ float Sl[2][kCombMaxD * kDeltaCols];
    const int s = blockIdx.x, h = blockIdx.y, cb = blockIdx.z, tid = threadIdx.x;
    const int D = a.D, V = a.V, H = a.H;
    int g0 = 0;
    for (int q = 0; q < s; ++q) g0 += (a.seq_starts[q + 1] - a.seq_starts[q] + a.seg_tokens - 1) / a.seg_tokens;
    const int begin = a.seq_starts[s];
    const int n_seg = (a.seq_starts[s + 1] - begin + a.seg_tokens - 1) / a.seg_tokens;
    if (n_seg <= 0) return;
    const int slot = a.state_slots[s];
    const bool from_slot = slot >= 0 && slot < a.n_slots && a.positions[begin] != 0;
    const int jj = tid % kDeltaCols, ib = tid / kDeltaCols, j = cb * kDeltaCols + jj;
    const int64_t DD = static_cast<int64_t>(D) * D, DV = static_cast<int64_t>(D) * V;
    const float* S0 = a.state + static_cast<int64_t>(from_slot ? slot : 0) * a.state_stride + h * DV;
    for (int m = ib; m < kCombMaxD; m += 256 / kDeltaCols) {  // (rows past the head's last stay zero: they meet zeros of P)
        Sl[0][m * kDeltaCols + jj] = (from_slot && m < D && j < V) ? S0[static_cast<int64_t>(m) * V + j] : 0.0f;
        Sl[1][m * kDeltaCols + jj] = 0.0f;
    }
    const int nb = (D + kCombTile - 1) / kCombTile, per_seg = nb * nb;
    const int n_tiles = (n_seg - 1) * per_seg;
    constexpr int NPRE = kCombTile * kCombTile / 256;
    float pre[NPRE];
    auto fetch = [&](int T) {
        const int g = T / per_seg, ibk = (T % per_seg) / nb, mbk = T % nb;
        const float* P = seg_p + (static_cast<int64_t>(g0 + g) * H + h) * DD;
#pragma unroll
        for (int q = 0; q < NPRE; ++q) {
            const int e = tid + q * 256;
            const int i = ibk * kCombTile + e / kCombTile, m = mbk * kCombTile + e % kCombTile;
            const float val = P[static_cast<int64_t>(min(i, D - 1)) * D + min(m, D - 1)];
            pre[q] = (i < D && m < D) ? val : 0.0f;
        }
    };
    // a segment's own end, for the rows of block ibk of step g * nb + ibk; asked for one step ahead, like the tiles (the barriers
    // below wait for LDS only, so what is on its way from memory stays on its way)
    auto fetch_z = [&](int step, float (&z)[4]) {
        const int g = step / nb, ibk = step % nb;
        const bool live = g + 1 < n_seg;  // (a request's last segment has none)
        const float* Zg = seg_z + (static_cast<int64_t>(g0 + g) * H + h) * DV;
#pragma unroll
        for (int q = 0; q < 4; ++q) {
            const int i = ibk * kCombTile + ib + 16 * q;
            z[q] = (live && i < D && j < V) ? Zg[static_cast<int64_t>(i) * V + j] : 0.0f;
        }
    };
    float z_next[4];
    fetch_z(0, z_next);
    if (n_tiles > 0) fetch(0);
    __syncthreads();
    typedef __attribute__((ext_vector_type(4))) float f32x4;
    int cur = 0;
    for (int g = 0; g < n_seg; ++g) {
        float* Sg = seg_start + (static_cast<int64_t>(g0 + g) * H + h) * DV;
        const bool more = g + 1 < n_seg;
        for (int ibk = 0; ibk < nb; ++ibk) {
            float acc[4];
#pragma unroll
            for (int q = 0; q < 4; ++q) acc[q] = z_next[q];
            if (g * nb + ibk + 1 < n_seg * nb) fetch_z(g * nb + ibk + 1, z_next);
            if (more) {
                for (int mbk = 0; mbk < nb; ++mbk) {
                    const int T = (g * nb + ibk) * nb + mbk;
#pragma unroll
                    for (int q = 0; q < NPRE; ++q) {
                        const int e = tid + q * 256;
                        Pt[(e / kCombTile) * kCombStride + e % kCombTile] = pre[q];
                    }
                    lds_barrier();
                    if (T + 1 < n_tiles) fetch(T + 1);
                    const float* Sc = Sl[cur] + mbk * kCombTile * kDeltaCols + jj;
#pragma unroll 4
                    for (int c = 0; c < kCombTile; c += 4) {
                        float sv[4];
#pragma unroll
                        for (int e = 0; e < 4; ++e) sv[e] = Sc[(c + e) * kDeltaCols];
#pragma unroll
                        for (int q = 0; q < 4; ++q) {
                            const f32x4 p4 = *reinterpret_cast<const f32x4*>(Pt + (ib + 16 * q) * kCombStride + c);
#pragma unroll
                            for (int e = 0; e < 4; ++e) acc[q] += p4[e] * sv[e];
                        }
                    }
                    lds_barrier();  // (the next tile takes this one's place)
                }
            }
#pragma unroll
            for (int q = 0; q < 4; ++q) {
                const int i = ibk * kCombTile + ib + 16 * q;
                if (i < D) Sl[cur ^ 1][i * kDeltaCols + jj] = acc[q];
            }
        }
        if (j < V)
            for (int m = ib; m < D; m += 256 / kDeltaCols) Sg[static_cast<int64_t>(m) * V + j] = Sl[cur][m * kDeltaCols + jj];
        lds_barrier();
        cur ^= 1;
    }
}

// The same for D up to 64 on the matrix cores in 32-bit floats (v_mfma_f32_16x16x4_f32): a workgroup a (request, head, 16 columns),
// its wave w rows 16 w .. 16 w + 15. What the chain over segments waits for is the trip of each segment's P and Z from memory, not the
// arithmetic: a wave's operand of P goes straight into registers, kCombDepth segments ahead, and only S passes through LDS. In step q of
// the product the four groups of 16 lanes hold rows 16 g + q of S (g the group), so that a lane's entries of P are 16 in a row.
constexpr int kCombDepth = 4;
typedef __attribute__((ext_vector_type(4))) float comb_f32x4;

template <bool WHOLE>  // WHOLE: D = 64, P in pieces of four floats; otherwise entries past the matrix are read from inside and taken as zeros
static __global__ void __launch_bounds__(256)
delta_combine_mfma_kernel(DeltaSegments a, const float* __restrict__ seg_z, const float* __restrict__ seg_p, float* __restrict__ seg_start) {
    constexpr int kGroup = 16 * 16 + 16;  // floats of 16 rows of S, the next group's rows in other banks
    __shared__ float Sl[2][4 * kGroup];
    const int s = blockIdx.x, h = blockIdx.y, cb = blockIdx.z, tid = threadIdx.x, lane = tid % kWave, wave = tid / kWave;
    const int D = WHOLE ? 64 : a.D, V = a.V, H = a.H;
    int g0 = 0;
    for (int q = 0; q < s; ++q) g0 += (a.seq_starts[q + 1] - a.seq_starts[q] + a.seg_tokens - 1) / a.seg_tokens;
    const int begin = a.seq_starts[s];
    const int n_seg = (a.seq_starts[s + 1] - begin + a.seg_tokens - 1) / a.seg_tokens;
    if (n_seg <= 0) return;
    const int slot = a.state_slots[s];
    const bool from_slot = slot >= 0 && slot < a.n_slots && a.positions[begin] != 0;
    const int li = lane % 16, grp = lane / 16, j = cb * kDeltaCols + li, jc = min(j, V - 1);
    const int64_t DD = static_cast<int64_t>(D) * D, DV = static_cast<int64_t>(D) * V;
    const float* S0 = a.state + static_cast<int64_t>(from_slot ? slot : 0) * a.state_stride + h * DV;
    const int row_p = min(16 * wave + li, D - 1);      // this lane's row of P, columns 16 grp ..
    const bool row_in = 16 * wave + li < D;
    // a lane's part of the result: rows 16 wave + 4 grp + r, column j
    const int row_s = 16 * wave + 4 * grp;
    float p[kCombDepth][16], z[kCombDepth][4];
    auto fetch = [&](int g, float (&pp)[16], float (&zz)[4]) {
        const int64_t at = static_cast<int64_t>(g0 + min(g, n_seg - 1)) * H + h;  // (past the last one: read again, not used)
        const float* P = seg_p + at * DD + static_cast<int64_t>(row_p) * D;
        const float* Z = seg_z + at * DV;
        if constexpr (WHOLE) {
#pragma unroll
            for (int q4 = 0; q4 < 4; ++q4) {
                const comb_f32x4 v = *reinterpret_cast<const comb_f32x4*>(P + 16 * grp + 4 * q4);
#pragma unroll
                for (int e = 0; e < 4; ++e) pp[4 * q4 + e] = v[e];
            }
        } else {
#pragma unroll
            for (int q = 0; q < 16; ++q) pp[q] = P[min(16 * grp + q, D - 1)];
        }
#pragma unroll
        for (int r = 0; r < 4; ++r) zz[r] = Z[static_cast<int64_t>(min(row_s + r, D - 1)) * V + jc];
    };
    // (entries past the matrix are made zeros where they are used: a choice beside a load would wait for that load alone)
    auto row_or_zero = [&](float v, int r) { return WHOLE || row_s + r < D ? v : 0.0f; };
    auto p_or_zero = [&](float v, int q) { return WHOLE || (row_in && 16 * grp + q < D) ? v : 0.0f; };
#pragma unroll
    for (int u = 0; u < kCombDepth; ++u) fetch(u, p[u], z[u]);
    float S[4];
#pragma unroll
    for (int r = 0; r < 4; ++r) S[r] = S0[static_cast<int64_t>(min(row_s + r, D - 1)) * V + jc];
    settle_loads(S);
#pragma unroll
    for (int r = 0; r < 4; ++r) S[r] = from_slot && row_s + r < D ? S[r] : 0.0f;  // (columns past the last one meet no other and are not kept)
    for (int gb = 0; gb < n_seg; gb += kCombDepth) {
#pragma unroll
        for (int u = 0; u < kCombDepth; ++u) {
            const int g = gb + u;
            if (g >= n_seg) break;  // (the same for the whole workgroup)
            float* out = seg_start + (static_cast<int64_t>(g0 + g) * H + h) * DV;
            if (j < V) {
#pragma unroll
                for (int r = 0; r < 4; ++r)
                    if (row_s + r < D) out[static_cast<int64_t>(row_s + r) * V + j] = S[r];
            }
            if (g + 1 >= n_seg) break;
            float* buf = Sl[g & 1];
#pragma unroll
            for (int r = 0; r < 4; ++r) buf[wave * kGroup + (4 * grp + r) * 16 + li] = S[r];
            lds_barrier();  // (one a segment: the buffer written two segments ago has been read by then)
            float b[16];
#pragma unroll
            for (int q = 0; q < 16; ++q) b[q] = buf[grp * kGroup + q * 16 + li];
            comb_f32x4 acc0 = {row_or_zero(z[u][0], 0), row_or_zero(z[u][1], 1), row_or_zero(z[u][2], 2), row_or_zero(z[u][3], 3)}, acc1 = {0.0f, 0.0f, 0.0f, 0.0f};
#pragma unroll
            for (int q = 0; q < 16; q += 2) {
                acc0 = __builtin_amdgcn_mfma_f32_16x16x4f32(p_or_zero(p[u][q], q), b[q], acc0, 0, 0, 0);
                acc1 = __builtin_amdgcn_mfma_f32_16x16x4f32(p_or_zero(p[u][q + 1], q + 1), b[q + 1], acc1, 0, 0, 0);
            }
#pragma unroll
            for (int r = 0; r < 4; ++r) S[r] = acc0[r] + acc1[r];
            fetch(g + kCombDepth, p[u], z[u]);
        }
    }
}

// Leaves in seg_start [segments][H][D][V] the state each segment of a step starts from, given every segment's Z and P.
inline void combine_segments(const DeltaSegments& a, const float* seg_z, const float* seg_p, float* seg_start, hipStream_t stream) {
    const dim3 grid(a.n_seqs, a.H, (a.V + kDeltaCols - 1) / kDeltaCols);
    if (a.D == 64) delta_combine_mfma_kernel<true><<<grid, 256, 0, stream>>>(a, seg_z, seg_p, seg_start);
    else if (a.D < 64) delta_combine_mfma_kernel<false><<<grid, 256, 0, stream>>>(a, seg_z, seg_p, seg_start);
    else delta_combine_kernel<<<grid, 256, 0, stream>>>(a, seg_z, seg_p, seg_start);
}

}  // namespace liyab
