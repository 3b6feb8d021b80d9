// A selective scan: a recurrence with a state of its own for every channel and state number,
//   S[c, n] <- exp(dt_c A[c, n]) S[c, n] + dt_c x_c B_n,    y_c = (sum_n S[c, n] C_n + D_c x_c) * silu(z_c),    A = -exp(A_log),
// where dt_c = softplus(Wdt low + bias), B and C are a token's own, from a projection of its x: rows [low: rank | B: N | C: N].
//
// liyab_scan_steps: the step sizes dt of a step's tokens. With bfloat16 weights the product runs on the matrix cores and `low`
//   enters it as two bfloat16 numbers a value, low = hi + lo (W hi + W lo: 16 bits of low), because a decay is multiplied by itself over hundreds of
//   tokens; with float weights as plain multiply-adds. Bias and softplus are 32-bit.
// liyab_selective_scan: the walk. A wave has 64 channels of a request's stretch of tokens, a lane a channel with its N states in
//   registers; a token's B and C are staged through LDS sixteen tokens at a time, x, dt and z are asked for eight tokens ahead. phase 0: a request's whole portion
//   by one wave. Long portions in segments side by side instead, in three launches: phase 1, every segment from zero for its end
//   state and the sum of its dt (the product of a segment's decays is exp(A sum dt)); phase 2, the segments of a
//   request strung together, which leaves the true state behind each; phase 3, every segment again from the state behind the one before it (a
//   request's first one from its slot), with outputs. The grids follow from the step's rows and requests alone.
// liyab_selective_single: a step of single tokens, step sizes included, in one kernel: four waves a (request, 64 channels), each with a
//   quarter of the rank and a quarter of the states.
//
// A request's slot holds S as [N, channels] and behind it the last taps - 1 rows of the convolution's input (position p at ring
// place p % (taps - 1)), which the walk keeps for the next step: the convolution, which reads them, has run. The state counts as zero at
// position 0, whatever the slot holds. States, decays and sums are 32-bit; exp(v) is taken as 2^(v log2 e).
#include "common.h"
#include "launchers.h"

namespace liyab {

constexpr int SS_CHUNK = 16;  // tokens whose B and C are staged together
constexpr int SS_AHEAD = 8;   // tokens whose x, dt and z are asked for together
constexpr float kLog2e = 1.4426950408889634f;

__device__ __forceinline__ float ss_exp2(float v) { return __builtin_amdgcn_exp2f(v); }
__device__ __forceinline__ float ss_softplus(float z) { return z > 20.0f ? z : log1pf(expf(z)); }
// The same for results that end in 16 bits: ln(1 + e), e = exp(-|z|) in (0, 1], as its series where e is small (1 + e rounds its digits away), by the
// logarithm instruction elsewhere; within some units of 32-bit precision of the above.
__device__ __forceinline__ float ss_softplus_fast(float z) {
    const float e = ss_exp2(-fabsf(z) * kLog2e);
    float s = fmaf(e, -0.125f, 1.0f / 7.0f);
    s = fmaf(s, e, -1.0f / 6.0f);
    s = fmaf(s, e, 0.2f);
    s = fmaf(s, e, -0.25f);
    s = fmaf(s, e, 1.0f / 3.0f);
    s = fmaf(s, e, -0.5f);
    s = fmaf(s, e, 1.0f) * e;
    const float l = __builtin_amdgcn_logf(1.0f + e) * 0.6931471805599453f;
    return fmaxf(z, 0.0f) + (e < 0.125f ? s : l);
}
__device__ __forceinline__ float ss_silu(float z) { return z / (1.0f + expf(-z)); }

typedef __attribute__((ext_vector_type(8))) __bf16 ss_bf16x8;
typedef __attribute__((ext_vector_type(16))) float ss_floatx16;
typedef __attribute__((ext_vector_type(4))) uint32_t ss_u32x4;

// a wave 32 tokens x 32 channels, straight from global memory in pieces of eight k; A: lane's row li, k 8 (lane / 32) .. + 7 of each 16. The
// weights' rows are ldw long, a multiple of 8, zeros behind the rank; what low holds behind its rank is read and masked.
__global__ void __launch_bounds__(256)
scan_steps_mfma_kernel(float* __restrict__ dt, const float* __restrict__ low, int64_t ldl, const bf16_t* __restrict__ w, int ldw, const float* __restrict__ bias,
                       int n, int C, int rank) {
    const int lane = threadIdx.x % 64, wave = threadIdx.x / 64;
    const int li = lane % 32, lk = (lane / 32) * 8;
    const int t0 = (blockIdx.y * 4 + wave) * 32, c0 = blockIdx.x * 32;
    if (t0 >= n) return;
    const float* lrow = low + static_cast<int64_t>(min(t0 + li, n - 1)) * ldl;
    const bf16_t* wrow = w + static_cast<int64_t>(min(c0 + li, C - 1)) * ldw;
    ss_floatx16 acc;
#pragma unroll
    for (int r = 0; r < 16; ++r) acc[r] = 0.0f;
    for (int k0 = 0; k0 < rank; k0 += 16) {
        union { ss_bf16x8 v; ss_u32x4 u; bf16_t e[8]; } fw, hi, lo;
        const int k = min(k0 + lk, ldw - 8);  // (a piece past the last one: the last one, masked)
        const f32x4_t a = *reinterpret_cast<const f32x4_t*>(lrow + k), b = *reinterpret_cast<const f32x4_t*>(lrow + k + 4);
        fw.u = *reinterpret_cast<const ss_u32x4*>(wrow + k);
#pragma unroll
        for (int e = 0; e < 8; ++e) {
            const float v = k0 + lk + e < rank ? (e < 4 ? a[e] : b[e - 4]) : 0.0f;
            hi.e[e] = float_to_bf16(v);
            lo.e[e] = float_to_bf16(v - bf16_to_float(hi.e[e]));
        }
        acc = __builtin_amdgcn_mfma_f32_32x32x16_bf16(hi.v, fw.v, acc, 0, 0, 0);
        acc = __builtin_amdgcn_mfma_f32_32x32x16_bf16(lo.v, fw.v, acc, 0, 0, 0);
    }
    // a lane holds channel li; token rows 8 (r / 4) + 4 (lane / 32) + r % 4
    const int c = c0 + li;
    if (c >= C) return;
    const float b = bias[c];
#pragma unroll
    for (int r = 0; r < 16; ++r) {
        const int t = t0 + 8 * (r / 4) + 4 * (lane / 32) + r % 4;
        if (t < n) dt[static_cast<int64_t>(t) * C + c] = ss_softplus_fast(acc[r] + b);
    }
}

__global__ void __launch_bounds__(256)
scan_steps_plain_kernel(float* __restrict__ dt, const float* __restrict__ low, int64_t ldl, const float* __restrict__ w, int ldw,
                        const float* __restrict__ bias, int C, int rank) {
    const int t = blockIdx.y, c = blockIdx.x * 256 + threadIdx.x;
    if (c >= C) return;
    const float* lrow = low + static_cast<int64_t>(t) * ldl;
    const float* wrow = w + static_cast<int64_t>(c) * ldw;
    float acc = 0.0f;
    for (int k = 0; k < rank; ++k) acc = fmaf(lrow[k], wrow[k], acc);
    dt[static_cast<int64_t>(t) * C + c] = ss_softplus(acc + bias[c]);
}

struct SelectiveArgs {
    void* out;        // [n, C] in the compute type
    const void* x;    // [n, C] in the compute type
    const float* dt;  // [n, C]
    const float* bc;  // B of token t at bc + t * ldb, C behind it
    int64_t ldb;
    const float* z;   // rows of ldz floats
    int64_t ldz;
    const float* a2;  // [N, C]: A log2 e
    const float* skip;
    float* state;
    int64_t state_stride;
    int n_slots;
    const float* raw;  // the convolution's input rows, of which the last `places` are kept
    int64_t ldr;
    int places;
    const int *seq_starts, *positions, *state_slots;
    int n_seqs, C, N, phase, seg_tokens, max_segs;
    float* seg_state;  // [segments][N][C]
    float* seg_dt;     // [segments][C]
};

// the last `places` rows of a request's convolution input (channel c) to their places in the ring behind the states
__device__ __forceinline__ void ss_keep(const SelectiveArgs& a, float* slot_base, int begin, int end, int c) {
    float* ring = slot_base + static_cast<int64_t>(a.N) * a.C;
    for (int t = max(begin, end - a.places); t < end; ++t) ring[static_cast<int64_t>(a.positions[t] % a.places) * a.C + c] = a.raw[static_cast<int64_t>(t) * a.ldr + c];
}

// the walk of tokens t0 .. t1 - 1 from S; kOut: with outputs, otherwise the sum of dt is returned
template <typename T, int NREG, bool kOut>
__device__ __forceinline__ float ss_walk(const SelectiveArgs& a, float (&S)[NREG], const float (&A2)[NREG], float skip, int t0, int t1, int cc, bool c_ok,
                                         float (&lb)[SS_CHUNK * NREG], float (&lc)[kOut ? SS_CHUNK * NREG : 1]) {
    const int lane = threadIdx.x;
    const T* x = static_cast<const T*>(a.x);
    T* out = static_cast<T*>(a.out);
    float px[SS_AHEAD], pd[SS_AHEAD], pz[SS_AHEAD];
    auto fetch = [&](int from) {  // (past the last token: the last one once more, never used)
#pragma unroll
        for (int j = 0; j < SS_AHEAD; ++j) {
            const int64_t t = min(from + j, t1 - 1);
            px[j] = to_float<T>(x[t * a.C + cc]);
            pd[j] = a.dt[t * a.C + cc];
            if constexpr (kOut) pz[j] = a.z[t * a.ldz + cc];
        }
    };
    float sum_dt = 0.0f;
    fetch(t0);
    for (int base = t0; base < t1; base += SS_CHUNK) {
        __syncthreads();  // (a workgroup is one wave: what was staged before has been read)
        for (int e = lane; e < SS_CHUNK * NREG; e += 64) {
            const int tt = e / NREG, i = e % NREG;
            const float* row = a.bc + static_cast<int64_t>(min(base + tt, t1 - 1)) * a.ldb;
            const int at = min(i, a.N - 1);
            const float b = row[at];
            lb[e] = i < a.N ? b : 0.0f;
            if constexpr (kOut) {
                const float q = row[a.N + at];
                lc[e] = i < a.N ? q : 0.0f;
            }
        }
        __syncthreads();
#pragma unroll
        for (int half = 0; half < SS_CHUNK / SS_AHEAD; ++half) {
            const int from = base + half * SS_AHEAD;
            if (from >= t1) break;
            float cx[SS_AHEAD], cd[SS_AHEAD], cz[SS_AHEAD];
#pragma unroll
            for (int j = 0; j < SS_AHEAD; ++j) {
                cx[j] = px[j];
                cd[j] = pd[j];
                if constexpr (kOut) cz[j] = pz[j];
            }
            fetch(from + SS_AHEAD);
#pragma unroll
            for (int j = 0; j < SS_AHEAD; ++j) {
                if (from + j < t1) {  // (the same for every lane)
                    const float* bt = lb + (half * SS_AHEAD + j) * NREG;
                    const float dx = cd[j] * cx[j];
                    float y0 = 0.0f, y1 = 0.0f;
#pragma unroll
                    for (int i = 0; i < NREG; ++i) {
                        S[i] = fmaf(ss_exp2(cd[j] * A2[i]), S[i], dx * bt[i]);
                        if constexpr (kOut) {
                            const float q = lc[(half * SS_AHEAD + j) * NREG + i];
                            if (i % 2) y1 = fmaf(S[i], q, y1);
                            else y0 = fmaf(S[i], q, y0);
                        }
                    }
                    if constexpr (kOut) {
                        const float y = fmaf(skip, cx[j], y0 + y1) * ss_silu(cz[j]);
                        if (c_ok) out[static_cast<int64_t>(from + j) * a.C + cc] = from_float<T>(y);
                    } else {
                        sum_dt += cd[j];
                    }
                }
            }
        }
    }
    return sum_dt;
}

// Segment g of a step in the order of its requests, found by a wave: its request s, the request's rows, and which of the request's segments it is; a lane
// a request, the running sum over the lanes. False past the last segment.
__device__ __forceinline__ bool ss_find(const int* __restrict__ seq_starts, int n_seqs, int seg_tokens, int g, int& s, int& begin, int& end, int& local) {
    const int lane = threadIdx.x % kWave;
    int before = 0;
    for (int base = 0; base < n_seqs; base += kWave) {
        const int i = min(base + lane, n_seqs - 1);
        const int b = seq_starts[i], e = seq_starts[i + 1];
        const int count = base + lane < n_seqs ? (e - b + seg_tokens - 1) / seg_tokens : 0;
        int sum = count;
#pragma unroll
        for (int o = 1; o < kWave; o *= 2) {
            const int v = __shfl_up(sum, o, kWave);
            if (lane >= o) sum += v;
        }
        const uint64_t past = __ballot(before + sum > g);
        if (past != 0) {
            const int l = __builtin_ctzll(past);
            s = base + l;
            begin = __builtin_amdgcn_readlane(b, l);
            end = __builtin_amdgcn_readlane(e, l);
            local = g - before - (__builtin_amdgcn_readlane(sum, l) - __builtin_amdgcn_readlane(count, l));
            return true;
        }
        before += __builtin_amdgcn_readlane(sum, kWave - 1);
    }
    return false;
}

template <typename T, int NREG, int PHASE>
__global__ void __launch_bounds__(64)
selective_scan_kernel(SelectiveArgs a) {
    constexpr bool kOut = PHASE != 1;
    __shared__ __attribute__((aligned(16))) float lb[SS_CHUNK * NREG];
    __shared__ __attribute__((aligned(16))) float lc[kOut ? SS_CHUNK * NREG : 1];
    const int c = blockIdx.x * 64 + threadIdx.x;
    const bool c_ok = c < a.C;
    const int cc = c_ok ? c : a.C - 1;  // a lane past the channels walks the last one along; nothing of it is stored
    int s = blockIdx.y, begin, end, t0 = 0, t1 = 0;
    bool last = true;
    if constexpr (PHASE == 0) {
        begin = t0 = a.seq_starts[s];
        end = t1 = a.seq_starts[s + 1];
        if (end <= begin) return;
    } else {
        int g;
        if (!ss_find(a.seq_starts, a.n_seqs, a.seg_tokens, blockIdx.y, s, begin, end, g)) return;  // a workgroup past the last segment
        t0 = begin + g * a.seg_tokens;
        t1 = min(t0 + a.seg_tokens, end);
        last = t1 == end;
        if (PHASE == 1 && last) return;  // (nobody needs the end state of a request's last segment from zero)
    }
    const int slot = a.state_slots[s];
    const bool slot_ok = slot >= 0 && slot < a.n_slots;
    float* base = a.state + static_cast<int64_t>(slot_ok ? slot : 0) * a.state_stride;
    float* seg = a.seg_state + static_cast<int64_t>(blockIdx.y) * a.N * a.C;  // (read or written in phases 1 and 3 only)
    const bool first = PHASE != 1 && t0 == begin;  // starts from the request's own state
    const bool from_slot = first && slot_ok && a.positions[begin] > 0;
    float S[NREG], A2[NREG];
#pragma unroll
    for (int i = 0; i < NREG; ++i) {
        // (a register past the last state holds that state once more: its B and C are staged as zeros)
        A2[i] = a.a2[static_cast<int64_t>(min(i, a.N - 1)) * a.C + cc];
        S[i] = 0.0f;
    }
    if ((PHASE == 3 && !first) || from_slot) {
        const float* src = first ? base : seg - static_cast<int64_t>(a.N) * a.C;  // (the segment before holds the state behind it)
#pragma unroll
        for (int i = 0; i < NREG; ++i) S[i] = src[static_cast<int64_t>(min(i, a.N - 1)) * a.C + cc];
    }
    const float sum_dt = ss_walk<T, NREG, kOut>(a, S, A2, kOut ? a.skip[cc] : 0.0f, t0, t1, cc, c_ok, lb, lc);
    if (!c_ok) return;
    if constexpr (PHASE == 1) {
#pragma unroll
        for (int i = 0; i < NREG; ++i)
            if (i < a.N) seg[static_cast<int64_t>(i) * a.C + c] = S[i];
        a.seg_dt[static_cast<int64_t>(blockIdx.y) * a.C + c] = sum_dt;
    } else if (last && slot_ok) {
#pragma unroll
        for (int i = 0; i < NREG; ++i)
            if (i < a.N) base[static_cast<int64_t>(i) * a.C + c] = S[i];
        if (a.places > 0) ss_keep(a, base, begin, end, c);
    }
}

// phase 2: a thread a (channel, state) of a request strings its segments together, where it has more than one; eight segments' ends are asked for together
__global__ void __launch_bounds__(256)
selective_combine_kernel(SelectiveArgs a) {
    const int s = blockIdx.y, begin = a.seq_starts[s];
    const int n_seg = (a.seq_starts[s + 1] - begin + a.seg_tokens - 1) / a.seg_tokens;
    if (n_seg <= 1) return;  // (its only segment starts from the slot)
    // the segments of the requests before this one, a lane a request
    int g0 = 0;
    for (int i = threadIdx.x % kWave; i < s; i += kWave) g0 += (a.seq_starts[i + 1] - a.seq_starts[i] + a.seg_tokens - 1) / a.seg_tokens;
#pragma unroll
    for (int o = 1; o < kWave; o *= 2) g0 += __shfl_xor(g0, o, kWave);
    const int64_t e = static_cast<int64_t>(blockIdx.x) * 256 + threadIdx.x;
    const int64_t NC = static_cast<int64_t>(a.N) * a.C;
    if (e >= NC) return;
    const int slot = a.state_slots[s], c = static_cast<int>(e % a.C);
    const bool slot_ok = slot >= 0 && slot < a.n_slots;
    float S = (slot_ok && a.positions[begin] > 0) ? a.state[static_cast<int64_t>(slot) * a.state_stride + e] : 0.0f;
    const float a2 = a.a2[e];
    float* st = a.seg_state + g0 * NC + e;
    const float* sd = a.seg_dt + static_cast<int64_t>(g0) * a.C + c;
    for (int g = 0; g < n_seg - 1; g += 8) {
        float end[8], sum[8];
#pragma unroll
        for (int j = 0; j < 8; ++j) {
            const int64_t gg = min(g + j, n_seg - 2);  // (the last segment's end is not written and not used)
            end[j] = st[gg * NC];
            sum[j] = sd[gg * a.C];
        }
        settle_loads(end);
        settle_loads(sum);
#pragma unroll
        for (int j = 0; j < 8; ++j) {
            if (g + j < n_seg - 1) {
                S = fmaf(ss_exp2(sum[j] * a2), S, end[j]);
                st[(g + j) * NC] = S;
            }
        }
    }
}

// one token a request
template <typename T>
__global__ void __launch_bounds__(256)
selective_single_kernel(SelectiveArgs a, const T* __restrict__ wt, const float* __restrict__ bias, int rank) {
    __shared__ float part[4][64], steps[64];
    const int lane = threadIdx.x % 64, wave = threadIdx.x / 64;
    const int s = blockIdx.y;
    const int c = blockIdx.x * 64 + lane;
    const bool c_ok = c < a.C;
    const int cc = c_ok ? c : a.C - 1;
    const int64_t t = a.seq_starts[s];
    const int slot = a.state_slots[s];
    const bool slot_ok = slot >= 0 && slot < a.n_slots;
    float* base = a.state + static_cast<int64_t>(slot_ok ? slot : 0) * a.state_stride;
    const int pos = a.positions[t];
    const bool from_slot = slot_ok && pos > 0;
    const float* row = a.bc + t * a.ldb;  // [low | B | C]
    const float x = to_float<T>(static_cast<const T*>(a.x)[t * a.C + cc]);
    // this wave's quarter of the states: the first four are asked for before anything is computed
    const int nq = (a.N + 3) / 4, n0 = wave * nq, n1 = min(a.N, n0 + nq);
    float S[4], A2[4];
    auto states = [&](int i0) {
#pragma unroll
        for (int j = 0; j < 4; ++j) {
            const int64_t at = static_cast<int64_t>(min(i0 + j, a.N - 1)) * a.C + cc;
            A2[j] = a.a2[at];
            S[j] = base[at];
        }
    };
    states(n0);
    const float z = a.z[t * a.ldz + cc], raw = a.places > 0 ? a.raw[t * a.ldr + cc] : 0.0f;
    // this wave's quarter of the rank; weights [rank, C], a row's channels side by side
    const int kq = (rank + 3) / 4, k1 = min(rank, (wave + 1) * kq);
    float acc = 0.0f;
    for (int k = wave * kq; k < k1; k += 16) {  // sixteen weights and the row's numbers beside them are asked for together (past the quarter: its last, times zero)
        float w[16], r[16];
#pragma unroll
        for (int j = 0; j < 16; ++j) {
            const int kk = min(k + j, k1 - 1);
            w[j] = to_float<T>(wt[static_cast<int64_t>(kk) * a.C + cc]);
            r[j] = row[kk];
        }
        settle_loads(w);
#pragma unroll
        for (int j = 0; j < 16; ++j) acc = fmaf(k + j < k1 ? r[j] : 0.0f, w[j], acc);
    }
    part[wave][lane] = acc;
    __syncthreads();
    if (wave == 0) steps[lane] = ss_softplus((part[0][lane] + part[1][lane]) + (part[2][lane] + part[3][lane]) + bias[cc]);
    __syncthreads();
    const float dt = steps[lane], dx = dt * x;
    float y = 0.0f;
    for (int i0 = n0; i0 < n1; i0 += 4) {
        if (i0 > n0) states(i0);
#pragma unroll
        for (int j = 0; j < 4; ++j) {
            const int i = i0 + j;
            if (i < n1) {
                const float v = fmaf(ss_exp2(dt * A2[j]), from_slot ? S[j] : 0.0f, dx * row[rank + i]);
                y = fmaf(v, row[rank + a.N + i], y);
                if (c_ok && slot_ok) base[static_cast<int64_t>(i) * a.C + c] = v;
            }
        }
    }
    part[wave][lane] = y;
    __syncthreads();
    if (wave == 0 && c_ok) {
        const float sum = (part[0][lane] + part[1][lane]) + (part[2][lane] + part[3][lane]);
        static_cast<T*>(a.out)[t * a.C + c] = from_float<T>(fmaf(a.skip[c], x, sum) * ss_silu(z));
        if (slot_ok && a.places > 0) base[static_cast<int64_t>(a.N) * a.C + static_cast<int64_t>(pos % a.places) * a.C + c] = raw;
    }
}

template <typename T, int NREG>
void launch_selective(const SelectiveArgs& a, hipStream_t stream) {
    const int cb = (a.C + 63) / 64;
    if (a.phase == 0) selective_scan_kernel<T, NREG, 0><<<dim3(cb, a.n_seqs), 64, 0, stream>>>(a);
    else if (a.phase == 1) selective_scan_kernel<T, NREG, 1><<<dim3(cb, a.max_segs), 64, 0, stream>>>(a);
    else selective_scan_kernel<T, NREG, 3><<<dim3(cb, a.max_segs), 64, 0, stream>>>(a);
}
template <typename T>
void launch_selective_any(const SelectiveArgs& a, hipStream_t stream) {
    if (a.N <= 4) launch_selective<T, 4>(a, stream);
    else if (a.N <= 8) launch_selective<T, 8>(a, stream);
    else if (a.N <= 16) launch_selective<T, 16>(a, stream);
    else if (a.N <= 24) launch_selective<T, 24>(a, stream);
    else if (a.N <= 32) launch_selective<T, 32>(a, stream);
    else if (a.N <= 64) launch_selective<T, 64>(a, stream);
    else launch_selective<T, 128>(a, stream);
}

}  // namespace liyab

using namespace liyab;

constexpr int kMaxScanStates = 128;

// dt: float [n, C]; low: float rows [n, ldl], `rank` of them used; w: rows of ldw in `dtype`, the first `rank` of [C, ldw] used, for bfloat16 zeros behind them
// and ldw a multiple of 8 that ldl (a multiple of 4) holds; bias: float [C].
extern "C" int liyab_scan_steps(float* dt, const float* low, int64_t ldl, const void* w, int ldw, int dtype, const float* bias, int n, int C, int rank,
                                hipStream_t stream) {
    LIYAB_REQUIRE(dt && low && w && bias, "scan_steps: null pointer");
    LIYAB_REQUIRE(n >= 0 && n <= 65535 && C > 0 && rank > 0 && ldl >= rank && ldw >= rank, "scan_steps: bad sizes n=%d C=%d rank=%d", n, C, rank);
    LIYAB_REQUIRE(dtype == kF32 || dtype == kBF16, "scan_steps: unknown dtype %d", dtype);
    LIYAB_REQUIRE(dtype == kF32 || (ldw % 8 == 0 && ldl % 4 == 0 && ldl >= ldw && (reinterpret_cast<uintptr_t>(low) & 15) == 0 && (reinterpret_cast<uintptr_t>(w) & 15) == 0),
                  "scan_steps: rows of %lld floats and weights of %d a row are not taken in 16-byte pieces", static_cast<long long>(ldl), ldw);
    if (n == 0) return 0;
    if (dtype == kF32)
        scan_steps_plain_kernel<<<dim3((C + 255) / 256, n), 256, 0, stream>>>(dt, low, ldl, static_cast<const float*>(w), ldw, bias, C, rank);
    else
        scan_steps_mfma_kernel<<<dim3((C + 31) / 32, (n + 127) / 128), 256, 0, stream>>>(dt, low, ldl, static_cast<const bf16_t*>(w), ldw, bias, n, C, rank);
    return check_launch("scan_steps");
}

// out, x [rows, C] in `dtype`; dt: float [rows, C]; bc: float rows of ldb, B [N] and behind it C [N]; z: float rows of ldz; a2: float [N, C]; skip: float
// [C]; state: float [n_slots, state_stride], S [N, C] and behind it the ring of `places` rows of raw (float rows of ldr). segments: 0,
// or the tokens a segment with seg_state [max_segs, N, C] and seg_dt [max_segs, C], where max_segs holds every segment of the step.
extern "C" int liyab_selective_scan(void* out, int dtype, const void* x, const float* dt, const float* bc, int64_t ldb, const float* z, int64_t ldz,
                                    const float* a2, const float* skip, float* state, int64_t state_stride, int n_slots, const float* raw, int64_t ldr,
                                    int places, const int* seq_starts, const int* positions, const int* state_slots, int n_seqs, int C, int N,
                                    int seg_tokens, int max_segs, float* seg_state, float* seg_dt, hipStream_t stream) {
    LIYAB_REQUIRE(out && x && dt && bc && z && a2 && skip && state && seq_starts && positions && state_slots, "selective_scan: null pointer");
    LIYAB_REQUIRE(dtype == kF32 || dtype == kBF16, "selective_scan: unknown dtype %d", dtype);
    LIYAB_REQUIRE(n_seqs >= 0 && n_seqs <= 65535 && C > 0 && N > 0 && N <= kMaxScanStates && ldb >= 2 * N && ldz >= C && n_slots > 0 && places >= 0,
                  "selective_scan: bad sizes C=%d N=%d (up to %d states)", C, N, kMaxScanStates);
    LIYAB_REQUIRE(state_stride >= static_cast<int64_t>(N + places) * C && (places == 0 || (raw != nullptr && ldr >= C)), "selective_scan: the slot does not hold the states and %d rows", places);
    LIYAB_REQUIRE(seg_tokens == 0 || (seg_tokens > 0 && max_segs > 0 && max_segs <= 65535 && seg_state && seg_dt), "selective_scan: segments need their scratch");
    if (n_seqs == 0) return 0;
    SelectiveArgs a{out, x, dt, bc, ldb, z, ldz, a2, skip, state, state_stride, n_slots, raw, ldr, places, seq_starts, positions, state_slots,
                    n_seqs, C, N, 0, seg_tokens, max_segs, seg_state, seg_dt};
    auto walk = [&](int phase) {
        a.phase = phase;
        if (dtype == kF32) launch_selective_any<float>(a, stream);
        else launch_selective_any<bf16_t>(a, stream);
    };
    if (seg_tokens == 0) {
        walk(0);
        return check_launch("selective_scan");
    }
    walk(1);
    if (const int rc = check_launch("selective_scan (segments' ends)")) return rc;
    a.phase = 2;
    selective_combine_kernel<<<dim3(static_cast<unsigned>((static_cast<int64_t>(N) * C + 255) / 256), n_seqs), 256, 0, stream>>>(a);
    if (const int rc = check_launch("selective_scan (segments' starts)")) return rc;
    walk(3);
    return check_launch("selective_scan");
}

// As above for a step of single tokens (n_seqs rows, one a request); low: float rows of ldb, [low: rank | B: N | C: N]; wt [rank, C] in `dtype`.
extern "C" int liyab_selective_single(void* out, int dtype, const void* x, const float* low, int64_t ldb, int rank, const void* wt, const float* bias,
                                      const float* z, int64_t ldz, const float* a2, const float* skip, float* state, int64_t state_stride, int n_slots,
                                      const float* raw, int64_t ldr, int places, const int* seq_starts, const int* positions, const int* state_slots,
                                      int n_seqs, int C, int N, hipStream_t stream) {
    LIYAB_REQUIRE(out && x && low && wt && bias && z && a2 && skip && state && seq_starts && positions && state_slots, "selective_single: null pointer");
    LIYAB_REQUIRE(dtype == kF32 || dtype == kBF16, "selective_single: unknown dtype %d", dtype);
    LIYAB_REQUIRE(n_seqs >= 0 && n_seqs <= 65535 && C > 0 && N > 0 && rank > 0 && ldb >= rank + 2 * N && ldz >= C && n_slots > 0 && places >= 0, "selective_single: bad sizes C=%d N=%d rank=%d", C, N, rank);
    LIYAB_REQUIRE(state_stride >= static_cast<int64_t>(N + places) * C && (places == 0 || (raw != nullptr && ldr >= C)), "selective_single: the slot does not hold the states and %d rows", places);
    if (n_seqs == 0) return 0;
    const SelectiveArgs a{out, x, nullptr, low, ldb, z, ldz, a2, skip, state, state_stride, n_slots, raw, ldr, places, seq_starts, positions, state_slots,
                          n_seqs, C, N, 0, 0, 0, nullptr, nullptr};
    const dim3 grid((C + 63) / 64, n_seqs);
    if (dtype == kF32) selective_single_kernel<float><<<grid, 256, 0, stream>>>(a, static_cast<const float*>(wt), bias, rank);
    else selective_single_kernel<bf16_t><<<grid, 256, 0, stream>>>(a, static_cast<const bf16_t*>(wt), bias, rank);
    return check_launch("selective_single");
}
