// A gated delta rule with a short convolution on its inputs: a head's state S [D, V] decays by one number a token and its key's
// old content is replaced at a rate beta:
//   q, k, v = silu(conv(.)) a channel over time (taps inputs, the last the current row's; no bias, zeros before the start)
//   q, k of a head to length one, x / sqrt(sum(x^2) + key_eps); q times q_scale;  beta = sigmoid(b),  g = exp(-exp(A_log) softplus(a + dt_bias))
//   S <- g S;  S <- S + k (beta (v - S^T k))^T;  o = S^T q              (value head h uses the q and k of head h / (H / G))
// A row of `src` (a projection's 32-bit sums): [q, G * D | k, G * D | v, H * V | ...], and from it the gate's logits, b and a at columns of
// their own. A request's slot: the heads' matrices [H, D, V], and behind them a ring of `taps` places of the 2 G D + H V channels before
// the convolution, position p at place p % taps. One place more than the convolution reads: where every request brings one token, the
// new row goes to a place nobody reads in that step, so the kernel that reads the ring can write it.
//
// liyab_gated_delta_prepare: every token's vectors as the recurrence wants them, float [n, 2 G D + H V + 2 H] = [q | k | v | g | beta];
//   a wave a (block of tokens, head of q, k or v).
// liyab_gated_delta_scan: a workgroup a (request, head, 64 columns) walks the request's rows of the step in order: four lanes side by
//   side share a column, each with a quarter of its rows in registers; the sums over a column's rows (S^T k and S^T q) come through the
//   lanes' own data path; tokens' vectors go through LDS a chunk at a time, the next chunk fetched while this one is computed. The last
//   rows go to the ring here, after the kernel that reads it. Long portions run in segments side by side (delta_segments.h): A_t =
//   g (I - beta k k^T), the outer product beta k v^T.
// liyab_gated_delta_single: a step of single tokens in one kernel, a workgroup a (request, head): convolution, unit vectors, decay and
//   rate, the recurrence, the head's norm (a weight of a head's width), times silu of the gate's logits, rounded once.
#include "common.h"
#include "delta_segments.h"
#include "launchers.h"

namespace liyab {

constexpr int kGdMax = 256;      // the widest heads
constexpr int kGdMaxTaps = 16;

__device__ __forceinline__ float gd_sigmoid(float z) { return 1.0f / (1.0f + expf(-z)); }
__device__ __forceinline__ float gd_softplus(float z) { return z > 20.0f ? z : log1pf(expf(z)); }

struct GdPrepareArgs {
    float* prep;
    const float* src;
    int64_t ld;
    const float* cw;          // [taps, C]: a tap's channels side by side
    int taps;
    const float* ring;        // of slot 0
    int64_t state_stride;
    int n_slots;
    const float *a_log, *dt_bias;
    int b_off, a_off;
    float key_eps, q_scale;
    const int *tok_seq, *positions, *seq_starts, *state_slots;
    int n, H, G, D, V;
};

// A wave takes kGdTokens consecutive rows of the step for one head's channels: a channel's weights are read once, and a row once for
// all the tokens whose taps it is. What lies before a request's first row of the step (its ring, or nothing) is the exception.
// TAPS: the number of taps, or 0 for any number (each row then reads its own taps).
constexpr int kGdTokens = 8;

template <int TAPS>
__global__ void __launch_bounds__(256)
gated_delta_prepare_kernel(GdPrepareArgs a) {
    const int units = 2 * a.G + a.H, taps = TAPS > 0 ? TAPS : a.taps;
    const int lane = threadIdx.x % kWave;
    const int item = __builtin_amdgcn_readfirstlane(blockIdx.x * 4 + threadIdx.x / kWave);
    if (item >= (a.n + kGdTokens - 1) / kGdTokens * units) return;
    const int t0 = item / units * kGdTokens, unit = item % units;
    const int GD = a.G * a.D, C = 2 * GD + a.H * a.V;
    const bool is_v = unit >= 2 * a.G;
    const int width = is_v ? a.V : a.D;
    const int c0 = is_v ? 2 * GD + (unit - 2 * a.G) * a.V : unit * a.D;
    const int64_t pld = C + 2 * a.H;
    constexpr int NQ = kGdMax / kWave, BACK = TAPS > 0 ? TAPS - 1 : 0, ROWS = kGdTokens + BACK;
    float x[kGdTokens][NQ];
#pragma unroll
    for (int tt = 0; tt < kGdTokens; ++tt)
#pragma unroll
        for (int q = 0; q < NQ; ++q) x[tt][q] = 0.0f;
#pragma unroll
    for (int q = 0; q < NQ; ++q) {
        if (q * kWave >= width) break;  // (the same for the whole wave)
        const int i = lane + q * kWave, c = c0 + min(i, width - 1);
        float rows[ROWS], w[TAPS > 0 ? TAPS : 1];
        if (TAPS > 0) {
#pragma unroll
            for (int r = 0; r < ROWS; ++r) rows[r] = a.src[static_cast<int64_t>(min(max(t0 - BACK + r, 0), a.n - 1)) * a.ld + c];
#pragma unroll
            for (int jt = 0; jt < TAPS; ++jt) w[jt] = a.cw[static_cast<int64_t>(jt) * C + c];
        }
#pragma unroll
        for (int tt = 0; tt < kGdTokens; ++tt) {
            const int t = min(t0 + tt, a.n - 1);
            const int s = a.tok_seq[t], p = a.positions[t], begin = a.seq_starts[s];
            float acc = 0.0f;
            if (TAPS > 0 && t - BACK >= begin && p >= BACK) {  // (the same for the whole wave, as everything but the channel)
#pragma unroll
                for (int jt = 0; jt < TAPS; ++jt) acc = fmaf(w[jt], rows[tt + jt], acc);
            } else {
                const int slot = a.state_slots[s];
                const bool slot_ok = slot >= 0 && slot < a.n_slots;
                const float* ring = a.ring + static_cast<int64_t>(slot_ok ? slot : 0) * a.state_stride;  // (not followed with one tap)
                for (int jt = 0; jt < taps; ++jt) {
                    const int back = taps - 1 - jt;
                    if (p - back < 0) continue;
                    float v = 0.0f;
                    if (t - back >= begin) v = a.src[static_cast<int64_t>(t - back) * a.ld + c];
                    else if (slot_ok) v = ring[static_cast<int64_t>((p - back) % taps) * C + c];
                    acc = fmaf(a.cw[static_cast<int64_t>(jt) * C + c], v, acc);
                }
            }
            x[tt][q] = i < width ? acc * gd_sigmoid(acc) : 0.0f;
        }
    }
#pragma unroll
    for (int tt = 0; tt < kGdTokens; ++tt) {
        if (t0 + tt >= a.n) break;
        float f = 1.0f;
        if (!is_v) {
            float ss = 0.0f;
#pragma unroll
            for (int q = 0; q < NQ; ++q) ss = fmaf(x[tt][q], x[tt][q], ss);
            f = 1.0f / sqrtf(wave_sum(ss) + a.key_eps) * (unit < a.G ? a.q_scale : 1.0f);
        }
        float* o = a.prep + static_cast<int64_t>(t0 + tt) * pld;
#pragma unroll
        for (int q = 0; q < NQ; ++q) {
            const int i = lane + q * kWave;
            if (i < width) o[c0 + i] = x[tt][q] * f;
        }
    }
    if (is_v && lane < 2 * kGdTokens && t0 + lane / 2 < a.n) {  // decay and rate of the head, a token two lanes
        const int h = unit - 2 * a.G, t = t0 + lane / 2;
        const float* row = a.src + static_cast<int64_t>(t) * a.ld;
        float* o = a.prep + static_cast<int64_t>(t) * pld + C + h;
        if (lane % 2 == 0) o[0] = expf(-expf(a.a_log[h]) * gd_softplus(row[a.a_off + h] + a.dt_bias[h]));
        else o[a.H] = gd_sigmoid(row[a.b_off + h]);
    }
}

struct GdScanArgs {
    float* out;               // [n, H * V] float32
    const float* prep;        // [n, 2 G D + H V + 2 H]
    const float* src;         // the rows before the convolution, kept in the ring
    int64_t ld;
    int taps;
    float* state;
    int64_t state_stride;
    int n_slots;
    const int *seq_starts, *positions, *state_slots;
    int n_seqs, H, G, D, V;
    int seg_tokens, max_segs, phase;  // as in delta_rule.hip: 0 the whole portion in one walk; 1 each segment for Z and P; 3 each from its true start
    float *seg_state, *seg_trans, *seg_start;
};

// REG: rows a lane holds (D <= 4 * REG). OUT: outputs are written (not in the pass that only wants the segments' ends).
template <int REG, bool OUT>
__global__ void __launch_bounds__(kDeltaWaves * kWave)
gated_delta_scan_kernel(GdScanArgs a) {
    constexpr int DP = 4 * REG, T = kDeltaWaves * kWave, COLS = kDeltaWaves * kDeltaCols;
    constexpr int CH = DP >= 64 ? 1024 / DP : 16;   // tokens a chunk: 16, 16, 8, 4 for REG = 8, 16, 32, 64
    constexpr int ROW = 2 * DP + COLS;              // a token's k, q and this workgroup's columns of v
    constexpr int PER = CH * ROW, NPRE = PER / T;
    static_assert(PER % T == 0 && 2 * CH <= T, "a chunk is dealt evenly among the threads");
    __shared__ __attribute__((aligned(16))) float lds[2 * PER];
    __shared__ float gb_s[2][2 * CH];
    const int tid = threadIdx.x, lane = tid % kWave, wave = tid / kWave;
    const int D = a.D, V = a.V, H = a.H;
    const int n_z = (V + COLS - 1) / COLS, n_grp = a.phase == 1 ? n_z + (D + COLS - 1) / COLS : n_z;  // phase 1: Z's columns, then P's
    const int grp = blockIdx.x % n_grp, h = (blockIdx.x / n_grp) % H, item = blockIdx.x / (n_grp * H);
    int s = item, begin, end;
    bool last_seg = true;
    if (a.seg_tokens > 0) {
        if (!find_segment(a.seq_starts, a.n_seqs, a.seg_tokens, item, s, begin, end, last_seg)) return;
        if (a.phase == 1 && last_seg) return;  // (nobody needs the end of a request's last segment from zero)
    } else {
        begin = a.seq_starts[s];
        end = a.seq_starts[s + 1];
    }
    if (begin >= end) return;
    const bool homogeneous = grp >= n_z;  // the walk for P: no outer products, from the unit matrix
    const int width = homogeneous ? D : V;  // columns of the matrix walked
    const int j_base = (homogeneous ? grp - n_z : grp) * COLS;
    const int rb = lane % kDeltaSplit, jl = wave * kDeltaCols + lane / kDeltaSplit, j = j_base + jl;
    const int i0 = rb * REG;
    const int slot = a.state_slots[s];
    const bool slot_ok = slot >= 0 && slot < a.n_slots;
    const bool fresh = a.positions[begin] == 0;
    float* Sg = a.state + static_cast<int64_t>(slot_ok ? slot : 0) * a.state_stride + static_cast<int64_t>(h) * D * V;
    const int64_t seg_at = (static_cast<int64_t>(item) * H + h) * D * width;
    float* S_seg = (a.phase == 3 ? a.seg_start : homogeneous ? a.seg_trans : a.seg_state) + seg_at;  // (written in phase 1, read in phase 3)
    float S[REG];
    bool mine[REG];
#pragma unroll
    for (int ii = 0; ii < REG; ++ii) {
        mine[ii] = i0 + ii < D && j < width;
        if (a.phase == 0) S[ii] = (mine[ii] && slot_ok && !fresh) ? Sg[static_cast<int64_t>(i0 + ii) * V + j] : 0.0f;
        else if (a.phase == 3) S[ii] = mine[ii] ? S_seg[static_cast<int64_t>(i0 + ii) * V + j] : 0.0f;
        else S[ii] = (mine[ii] && homogeneous && i0 + ii == j) ? 1.0f : 0.0f;
    }
    const int GD = a.G * D, C = 2 * GD + H * V;
    const int64_t pld = C + 2 * H;
    const int hk = h / (H / a.G);
    // element e of a chunk: token e / ROW; of its row k (0 .. DP), q (DP .. 2 DP), v (the columns of this workgroup)
    float pre[NPRE], pre_gb = 0.0f;
    auto fetch = [&](int c0) {
#pragma unroll
        for (int q = 0; q < NPRE; ++q) {
            const int e = tid + q * T;
            const int tt = e / ROW, x = e % ROW;
            const float* row = a.prep + static_cast<int64_t>(min(c0 + tt, end - 1)) * pld;
            const bool is_v = x >= 2 * DP;
            const int i = is_v ? j_base + x - 2 * DP : x % DP;
            const int at = is_v ? 2 * GD + h * V + min(i, V - 1) : (x < DP ? GD : 0) + hk * D + min(i, D - 1);
            const float val = row[at];
            pre[q] = is_v ? (i < V && !homogeneous ? val : 0.0f) : (i < D ? val : 0.0f);
        }
        if (tid < 2 * CH) pre_gb = a.prep[static_cast<int64_t>(min(c0 + tid / 2, end - 1)) * pld + C + (tid % 2) * H + h];
    };
    auto stash = [&](int buf) {
#pragma unroll
        for (int q = 0; q < NPRE; ++q) lds[buf * PER + tid + q * T] = pre[q];
        if (tid < 2 * CH) gb_s[buf][tid] = pre_gb;
    };
    fetch(begin);
    stash(0);
    __syncthreads();
    int which = 0;
    for (int c0 = begin; c0 < end; c0 += CH) {
        const bool more = c0 + CH < end;
        if (more) fetch(c0 + CH);
        const float* buf = lds + which * PER;
        const int n_tok = min(CH, end - c0);
        for (int tt = 0; tt < n_tok; ++tt) {
            const float* k = buf + tt * ROW + i0;
            const float* r = k + DP;
            const float v = buf[tt * ROW + 2 * DP + jl];
            const float g = gb_s[which][2 * tt], beta = gb_s[which][2 * tt + 1];
            f32x4_t k4[REG / 4];
            f32x4_t seen4 = {0.0f, 0.0f, 0.0f, 0.0f};
#pragma unroll
            for (int q4 = 0; q4 < REG / 4; ++q4) {
                k4[q4] = *reinterpret_cast<const f32x4_t*>(k + 4 * q4);
#pragma unroll
                for (int e = 0; e < 4; ++e) seen4[e] = fmaf(k4[q4][e], S[4 * q4 + e], seen4[e]);  // (rows that are not this lane's hold zero)
            }
            const float seen = group_sum<kDeltaSplit>((seen4[0] + seen4[1]) + (seen4[2] + seen4[3]));
            const float u = beta * (v - g * seen);
            f32x4_t o4 = {0.0f, 0.0f, 0.0f, 0.0f};
#pragma unroll
            for (int q4 = 0; q4 < REG / 4; ++q4) {
                f32x4_t r4;
                if (OUT) r4 = *reinterpret_cast<const f32x4_t*>(r + 4 * q4);
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    S[4 * q4 + e] = fmaf(g, S[4 * q4 + e], k4[q4][e] * u);  // (k is zero past the head's last row)
                    if (OUT) o4[e] = fmaf(r4[e], S[4 * q4 + e], o4[e]);
                }
            }
            if (OUT) {
                const float o = group_sum<kDeltaSplit>((o4[0] + o4[1]) + (o4[2] + o4[3]));
                if (rb == 0 && j < V) a.out[static_cast<int64_t>(c0 + tt) * H * V + h * V + j] = o;
            }
        }
        if (more) stash(which ^ 1);
        __syncthreads();
        which ^= 1;
    }
    if (a.phase == 1) {
#pragma unroll
        for (int ii = 0; ii < REG; ++ii)
            if (mine[ii]) S_seg[static_cast<int64_t>(i0 + ii) * width + j] = S[ii];
    } else if (slot_ok && last_seg) {
#pragma unroll
        for (int ii = 0; ii < REG; ++ii)
            if (mine[ii]) Sg[static_cast<int64_t>(i0 + ii) * V + j] = S[ii];
        // the request's last taps - 1 rows to the ring, the channels dealt among the request's workgroups
        if (a.taps > 1) {
            float* ring = a.state + static_cast<int64_t>(slot) * a.state_stride + static_cast<int64_t>(H) * D * V;
            for (int t = max(a.seq_starts[s], end - (a.taps - 1)); t < end; ++t) {
                float* dst = ring + static_cast<int64_t>(a.positions[t] % a.taps) * C;
                for (int c = (h * n_grp + grp) * T + tid; c < C; c += H * n_grp * T) dst[c] = a.src[static_cast<int64_t>(t) * a.ld + c];
            }
        }
    }
}

struct GdSingleArgs {
    void* out;                // [n, H * V], the compute type
    const float* src;
    int64_t ld;
    const float* cw;
    int taps;
    const float *a_log, *dt_bias;
    int g_off, b_off, a_off;
    const float* norm_w;      // [V]
    float eps, key_eps, q_scale;
    float* state;
    int64_t state_stride;
    int n_slots;
    const int *seq_starts, *positions, *state_slots;
    int H, G, D, V;
};

template <typename OutT, int REG, int TAPS>
__global__ void __launch_bounds__(kDeltaWaves * kWave)
gated_delta_single_kernel(GdSingleArgs a) {
    constexpr int DP = 4 * REG, COLS = kDeltaWaves * kDeltaCols;
    __shared__ __attribute__((aligned(16))) float k_s[DP], q_s[DP];
    __shared__ float v_s[kGdMax], o_s[kGdMax], gb_s[2], red[kDeltaWaves];
    const int tid = threadIdx.x, lane = tid % kWave, wave = __builtin_amdgcn_readfirstlane(tid / kWave);
    const int h = blockIdx.x % a.H, s = blockIdx.x / a.H;
    const int t = s;  // (the host sends steps of single tokens only: as many rows as requests)
    const int p = a.positions[t], slot = a.state_slots[s];
    if (a.seq_starts[s] != s || a.seq_starts[s + 1] != s + 1) return;
    const int D = a.D, V = a.V, H = a.H, GD = a.G * D, C = 2 * GD + H * V;
    const int per_k = H / a.G, hk = h / per_k;
    const bool slot_ok = slot >= 0 && slot < a.n_slots;
    const bool old = slot_ok && p > 0;
    float* base = a.state + static_cast<int64_t>(slot_ok ? slot : 0) * a.state_stride;
    float* Sg = base + static_cast<int64_t>(h) * D * V;
    float* ring = base + static_cast<int64_t>(H) * D * V;
    const float* row = a.src + static_cast<int64_t>(t) * a.ld;
    const int rb = lane % kDeltaSplit, i0 = rb * REG, jl = wave * kDeltaCols + lane / kDeltaSplit;
    float S[REG];
    auto load = [&](int j) {  // places outside the matrix read one inside it, and are zeros after settle()
#pragma unroll
        for (int ii = 0; ii < REG; ++ii) S[ii] = Sg[static_cast<int64_t>(min(i0 + ii, D - 1)) * V + min(j, V - 1)];
    };
    auto settle = [&](int j) {
        settle_loads(S);
#pragma unroll
        for (int ii = 0; ii < REG; ++ii) S[ii] = (i0 + ii < D && j < V && old) ? S[ii] : 0.0f;
    };
    // The gate's logits and the norm's weights, which the last lines need, are asked for first, then what the vectors are made of, then
    // the first block of columns: it is on its way while the vectors are made.
    const float z = row[a.g_off + h * V + min(tid, V - 1)], norm_w = a.norm_w[min(tid, V - 1)];
    if (wave < 3) {
        // a wave a vector: k, q, v
        const int width = wave == 2 ? V : D, pad = wave == 2 ? V : DP;
        const int c0 = wave == 0 ? GD + hk * D : wave == 1 ? hk * D : 2 * GD + h * V;
        const int taps = TAPS > 0 ? TAPS : a.taps;
        const int here = p % taps;  // this row's place in the ring
        const bool writes = slot_ok && taps > 1 && (wave == 2 || h % per_k == 0);
        auto place = [&](int back) { return here - back + (here < back ? taps : 0); };
        constexpr int NQ = kGdMax / kWave;
        float x[NQ];
#pragma unroll
        for (int q = 0; q < NQ; ++q) x[q] = 0.0f;
        float ss = 0.0f;
#pragma unroll
        for (int q = 0; q < NQ; ++q) {
            if (q * kWave >= width) break;  // (the same for the whole wave)
            const int i = lane + q * kWave, c = c0 + min(i, width - 1);
            const float now = row[c];
            float acc = 0.0f;
            if constexpr (TAPS > 0) {
                // all of a channel's inputs and weights are asked for together
                float before[TAPS], w[TAPS];  // (the last input is this row's)
                before[TAPS - 1] = now;
#pragma unroll
                for (int jt = 0; jt < TAPS - 1; ++jt) before[jt] = ring[static_cast<int64_t>(place(TAPS - 1 - jt)) * C + c];
#pragma unroll
                for (int jt = 0; jt < TAPS; ++jt) w[jt] = a.cw[static_cast<int64_t>(jt) * C + c];
                if (q == 0) load(jl);
                settle_loads(before);
                settle_loads(w);
#pragma unroll
                for (int jt = 0; jt < TAPS; ++jt) acc = fmaf(w[jt], (slot_ok && p - (TAPS - 1 - jt) >= 0) || jt == TAPS - 1 ? before[jt] : 0.0f, acc);
            } else {
                if (q == 0) load(jl);
                for (int jt = 0; jt < taps - 1; ++jt) {
                    const int back = taps - 1 - jt;
                    const float before = ring[static_cast<int64_t>(place(back)) * C + c];
                    acc = fmaf(a.cw[static_cast<int64_t>(jt) * C + c], slot_ok && p - back >= 0 ? before : 0.0f, acc);
                }
                acc = fmaf(a.cw[static_cast<int64_t>(taps - 1) * C + c], now, acc);
            }
            x[q] = i < width ? acc * gd_sigmoid(acc) : 0.0f;
            ss = fmaf(x[q], x[q], ss);
            if (writes && i < width) ring[static_cast<int64_t>(here) * C + c] = now;
        }
        float f = 1.0f;
        if (wave < 2) f = 1.0f / sqrtf(wave_sum(ss) + a.key_eps) * (wave == 1 ? a.q_scale : 1.0f);
        float* dst = wave == 0 ? k_s : wave == 1 ? q_s : v_s;
#pragma unroll
        for (int q = 0; q < kGdMax / kWave; ++q) {
            const int i = lane + q * kWave;
            if (i < pad) dst[i] = x[q] * f;  // (zeros behind a key's or query's last entry)
        }
    } else {
        const float decay_in = row[a.a_off + h], rate_in = row[a.b_off + h], a_log = a.a_log[h], dt_bias = a.dt_bias[h];
        load(jl);
        if (lane == 0) {
            gb_s[0] = expf(-expf(a_log) * gd_softplus(decay_in + dt_bias));
            gb_s[1] = gd_sigmoid(rate_in);
        }
    }
    lds_barrier();  // (the state's columns may stay on their way, the ring's new row too)
    const float g = gb_s[0], beta = gb_s[1];
    float ss = 0.0f;
    for (int c0 = 0; c0 < V; c0 += COLS) {
        const int j = c0 + jl;
        if (c0 > 0) load(j);
        settle(j);
        f32x4_t seen4 = {0.0f, 0.0f, 0.0f, 0.0f};
#pragma unroll
        for (int q4 = 0; q4 < REG / 4; ++q4) {
            const f32x4_t k4 = *reinterpret_cast<const f32x4_t*>(k_s + i0 + 4 * q4);
#pragma unroll
            for (int e = 0; e < 4; ++e) seen4[e] = fmaf(k4[e], S[4 * q4 + e], seen4[e]);
        }
        const float seen = group_sum<kDeltaSplit>((seen4[0] + seen4[1]) + (seen4[2] + seen4[3]));
        const float u = beta * (v_s[min(j, V - 1)] - g * seen);
        f32x4_t o4 = {0.0f, 0.0f, 0.0f, 0.0f};
#pragma unroll
        for (int q4 = 0; q4 < REG / 4; ++q4) {
            const f32x4_t k4 = *reinterpret_cast<const f32x4_t*>(k_s + i0 + 4 * q4), r4 = *reinterpret_cast<const f32x4_t*>(q_s + i0 + 4 * q4);
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                S[4 * q4 + e] = fmaf(g, S[4 * q4 + e], k4[e] * u);
                o4[e] = fmaf(r4[e], S[4 * q4 + e], o4[e]);
            }
        }
        const float o = group_sum<kDeltaSplit>((o4[0] + o4[1]) + (o4[2] + o4[3]));
        if (rb == 0 && j < V) {
            o_s[j] = o;
            ss = fmaf(o, o, ss);
        }
        if (slot_ok) {
#pragma unroll
            for (int ii = 0; ii < REG; ++ii)
                if (i0 + ii < D && j < V) Sg[static_cast<int64_t>(i0 + ii) * V + j] = S[ii];
        }
    }
    ss = wave_sum(ss);
    if (lane == 0) red[wave] = ss;
    lds_barrier();
    const float rinv = 1.0f / sqrtf((red[0] + red[1] + red[2] + red[3]) / static_cast<float>(V) + a.eps);
    if (tid < V) static_cast<OutT*>(a.out)[(static_cast<int64_t>(t) * H + h) * V + tid] = from_float<OutT>(o_s[tid] * rinv * norm_w * z * gd_sigmoid(z));
}

}  // namespace liyab

using namespace liyab;

extern "C" int liyab_gated_delta_takes(int D, int V) { return D >= 1 && D <= kGdMax && V >= 1 && V <= kGdMax ? 1 : 0; }

static bool gd_sizes_ok(int64_t ld, int taps, int64_t state_stride, int n_slots, int H, int G, int D, int V) {
    if (H <= 0 || G <= 0 || H % G != 0 || !liyab_gated_delta_takes(D, V) || taps < 1 || taps > kGdMaxTaps || n_slots <= 0) return false;
    const int64_t C = 2 * static_cast<int64_t>(G) * D + static_cast<int64_t>(H) * V;
    return ld >= C && state_stride >= static_cast<int64_t>(H) * D * V + (taps > 1 ? taps * C : 0);
}

extern "C" int liyab_gated_delta_prepare(float* prep, const float* src, int64_t ld, const float* cw, int taps, const float* ring, int64_t state_stride,
                                         int n_slots, const float* a_log, const float* dt_bias, int b_off, int a_off, float key_eps, float q_scale,
                                         const int* tok_seq, const int* positions, const int* seq_starts, const int* state_slots, int n, int H, int G,
                                         int D, int V, hipStream_t stream) {
    LIYAB_REQUIRE(prep && src && cw && ring && a_log && dt_bias && tok_seq && positions && seq_starts && state_slots, "gated_delta_prepare: null pointer");
    LIYAB_REQUIRE(n >= 0 && gd_sizes_ok(ld, taps, state_stride, n_slots, H, G, D, V), "gated_delta_prepare: bad sizes H=%d G=%d D=%d V=%d taps=%d", H, G, D, V, taps);
    LIYAB_REQUIRE(b_off >= 0 && a_off >= 0 && b_off + H <= ld && a_off + H <= ld, "gated_delta_prepare: the rates' or decays' columns pass the rows");
    if (n == 0) return 0;
    const GdPrepareArgs a{prep, src, ld, cw, taps, ring, state_stride, n_slots, a_log, dt_bias, b_off, a_off, key_eps, q_scale,
                          tok_seq, positions, seq_starts, state_slots, n, H, G, D, V};
    const int64_t items = static_cast<int64_t>((n + kGdTokens - 1) / kGdTokens) * (2 * G + H);
    LIYAB_REQUIRE(items < (int64_t(1) << 31) - 4, "gated_delta_prepare: too many tokens");
    const unsigned grid = static_cast<unsigned>((items + 3) / 4);
    if (taps == 4) gated_delta_prepare_kernel<4><<<grid, 256, 0, stream>>>(a);
    else if (taps == 3) gated_delta_prepare_kernel<3><<<grid, 256, 0, stream>>>(a);
    else if (taps == 2) gated_delta_prepare_kernel<2><<<grid, 256, 0, stream>>>(a);
    else gated_delta_prepare_kernel<0><<<grid, 256, 0, stream>>>(a);
    return check_launch("gated_delta_prepare");
}

extern "C" int liyab_gated_delta_scan(float* out, const float* prep, const float* src, int64_t ld, int taps, float* state, int64_t state_stride,
                                      int n_slots, const int* seq_starts, const int* positions, const int* state_slots, int n_seqs, int H, int G,
                                      int D, int V, int seg_tokens, int max_segs, float* seg_state, float* seg_trans, float* seg_start,
                                      hipStream_t stream) {
    LIYAB_REQUIRE(out && prep && src && state && seq_starts && positions && state_slots, "gated_delta_scan: null pointer");
    LIYAB_REQUIRE(seg_tokens >= 0 && (seg_tokens == 0 || (max_segs > 0 && seg_state && seg_trans && seg_start)), "gated_delta_scan: segments need their count and scratch");
    LIYAB_REQUIRE(n_seqs >= 0 && gd_sizes_ok(ld, taps, state_stride, n_slots, H, G, D, V), "gated_delta_scan: bad sizes H=%d G=%d D=%d V=%d taps=%d", H, G, D, V, taps);
    if (n_seqs == 0) return 0;
    GdScanArgs a{out, prep, src, ld, taps, state, state_stride, n_slots, seq_starts, positions, state_slots, n_seqs, H, G, D, V,
                 seg_tokens, max_segs, 0, seg_state, seg_trans, seg_start};
    constexpr int COLS = kDeltaWaves * kDeltaCols, T = kDeltaWaves * kWave;
    const int n_z = (V + COLS - 1) / COLS, n_p = (D + COLS - 1) / COLS;
    auto walk = [&](const GdScanArgs& p, int64_t items, bool outputs) {
        const dim3 grid(static_cast<unsigned>(items * H * (p.phase == 1 ? n_z + n_p : n_z)));
        auto go = [&](auto reg) {
            constexpr int R = decltype(reg)::value;
            if (outputs) gated_delta_scan_kernel<R, true><<<grid, T, 0, stream>>>(p);
            else gated_delta_scan_kernel<R, false><<<grid, T, 0, stream>>>(p);
        };
        if (D <= 32) go(std::integral_constant<int, 8>{});
        else if (D <= 64) go(std::integral_constant<int, 16>{});
        else if (D <= 128) go(std::integral_constant<int, 32>{});
        else go(std::integral_constant<int, 64>{});
    };
    if (seg_tokens > 0) {
        GdScanArgs p = a;
        p.phase = 1;
        walk(p, max_segs, false);
        const DeltaSegments segs{state, state_stride, n_slots, seq_starts, positions, state_slots, n_seqs, H, D, V, seg_tokens};
        combine_segments(segs, seg_state, seg_trans, seg_start, stream);
        p.phase = 3;
        walk(p, max_segs, true);
        return check_launch("gated_delta_scan");
    }
    walk(a, n_seqs, true);
    return check_launch("gated_delta_scan");
}

extern "C" int liyab_gated_delta_single(void* out, int out_dtype, const float* src, int64_t ld, const float* cw, int taps, const float* a_log,
                                        const float* dt_bias, int g_off, int b_off, int a_off, const float* norm_w, float eps, float key_eps,
                                        float q_scale, float* state, int64_t state_stride, int n_slots, const int* seq_starts, const int* positions,
                                        const int* state_slots, int n_seqs, int H, int G, int D, int V, hipStream_t stream) {
    LIYAB_REQUIRE(out && src && cw && a_log && dt_bias && norm_w && state && seq_starts && positions && state_slots, "gated_delta_single: null pointer");
    LIYAB_REQUIRE(n_seqs >= 0 && gd_sizes_ok(ld, taps, state_stride, n_slots, H, G, D, V), "gated_delta_single: bad sizes H=%d G=%d D=%d V=%d taps=%d", H, G, D, V, taps);
    LIYAB_REQUIRE(g_off >= 0 && b_off >= 0 && a_off >= 0 && g_off + static_cast<int64_t>(H) * V <= ld && b_off + H <= ld && a_off + H <= ld,
                  "gated_delta_single: the gate's, rates' or decays' columns pass the rows");
    LIYAB_REQUIRE(out_dtype == kF32 || out_dtype == kBF16, "gated_delta_single: unknown dtype %d", out_dtype);
    if (n_seqs == 0) return 0;
    const GdSingleArgs a{out, src, ld, cw, taps, a_log, dt_bias, g_off, b_off, a_off, norm_w, eps, key_eps, q_scale, state, state_stride, n_slots,
                         seq_starts, positions, state_slots, H, G, D, V};
    const unsigned grid = static_cast<unsigned>(n_seqs) * static_cast<unsigned>(H);
    constexpr int T = kDeltaWaves * kWave;
    auto run = [&](auto zero) {
        using O = decltype(zero);
        auto sized = [&](auto nt) {
            constexpr int N = decltype(nt)::value;
            if (D <= 32) gated_delta_single_kernel<O, 8, N><<<grid, T, 0, stream>>>(a);
            else if (D <= 64) gated_delta_single_kernel<O, 16, N><<<grid, T, 0, stream>>>(a);
            else if (D <= 128) gated_delta_single_kernel<O, 32, N><<<grid, T, 0, stream>>>(a);
            else gated_delta_single_kernel<O, 64, N><<<grid, T, 0, stream>>>(a);
        };
        if (taps == 4) sized(std::integral_constant<int, 4>{});
        else sized(std::integral_constant<int, 0>{});
    };
    if (out_dtype == kF32) run(float{});
    else run(bf16_t{});
    return check_launch("gated_delta_single");
}
