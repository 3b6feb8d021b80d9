// The residual stream as several copies that learned weights mix (hyper-connections), or as one: the rows' update between two
// sublayers, together with what the next sublayer reads.
//
// liyab_streams_update, for each token (its S streams of d 32-bit floats lie side by side in x):
//   y    = the sum of the sublayer's n_sum rows of the token, in their order; where `ids` says -1 for one of the first n_ids of
//          them (a routed feed-forward's entry that took an identity expert), weights * h takes the place of a row: h are the rows the
//          sublayer read (they may lie where `out` goes: a thread reads its entries of them before it writes)
//   x_t <- sum_s mix[s, t] x_s + add[t] y          all streams from the old ones; without `mix`: x_t + add[t] y; without `add`: ones
//   u    = sum_s in[s] x_s of the new streams (without `in`: their plain sum)
//   out  = u / sqrt(mean(u^2) + eps) * w in the output type
// Every part is optional: `enter` (rows [n, d]) first sets all streams to those rows; without y the streams stay as they are;
// without `out` nothing is read off them; `rows` gathers (what is read off them only: the final norm of the wanted rows).
// All sums and the norm are 32-bit; a result is rounded once, to the output type.
#include "common.h"
#include "launchers.h"

namespace liyab {

constexpr int ST_THREADS = 256;
constexpr int ST_MAX_STREAMS = 8;
constexpr int ST_HELD = 4;  // groups of VEC entries of u a thread keeps between the two passes; wider rows are read again

struct StreamsArgs {
    float* x;
    const float* enter;
    const float* y;
    int n_sum, n_ids;
    const int* ids;
    const float* weights;
    const void* h;
    const float *mix, *add, *in, *w;
    float eps;
    void* out;
    const int* rows;
    int d;
};

template <int VEC>
struct StVec {
    float v[VEC];
};
template <int VEC>
__device__ __forceinline__ StVec<VEC> st_load(const float* p) {
    StVec<VEC> r;
    if constexpr (VEC == 4) {
        const f32x4_t q = *reinterpret_cast<const f32x4_t*>(p);
        r.v[0] = q[0]; r.v[1] = q[1]; r.v[2] = q[2]; r.v[3] = q[3];
    } else {
        r.v[0] = *p;
    }
    return r;
}

template <typename T, int S, int VEC>
__global__ void __launch_bounds__(ST_THREADS)
streams_update_kernel(StreamsArgs a) {
    __shared__ float red[ST_THREADS / kWave];
    const int t = blockIdx.x, d = a.d;
    const int64_t src = a.rows != nullptr ? a.rows[t] : t;
    float* xr = a.x + src * S * d;
    float mix[S][S], add[S], in[S];
#pragma unroll
    for (int s = 0; s < S; ++s) {
        add[s] = a.add != nullptr ? a.add[s] : 1.0f;
        in[s] = a.in != nullptr ? a.in[s] : 1.0f;
#pragma unroll
        for (int to = 0; to < S; ++to) mix[s][to] = a.mix != nullptr ? a.mix[s * S + to] : (s == to ? 1.0f : 0.0f);
    }
    const int groups = d / VEC;  // (VEC 4 only where d is a multiple of 4)
    auto streams_of = [&](int i, StVec<VEC> (&x)[S]) {
        if (a.enter != nullptr) {
            const StVec<VEC> e = st_load<VEC>(a.enter + src * d + i);
#pragma unroll
            for (int s = 0; s < S; ++s) x[s] = e;
        } else {
#pragma unroll
            for (int s = 0; s < S; ++s) x[s] = st_load<VEC>(xr + static_cast<int64_t>(s) * d + i);
        }
    };
    auto read_off = [&](const StVec<VEC> (&x)[S]) {
        StVec<VEC> u;
#pragma unroll
        for (int e = 0; e < VEC; ++e) {
            float v = in[0] * x[0].v[e];
#pragma unroll
            for (int s = 1; s < S; ++s) v = fmaf(in[s], x[s].v[e], v);
            u.v[e] = v;
        }
        return u;
    };
    // the new streams at entries i .. i + VEC - 1, written where they changed; what the next sublayer reads of them
    auto update = [&](int i) {
        StVec<VEC> x[S];
        streams_of(i, x);
        if (a.y != nullptr) {
            const float* yr = a.y + src * a.n_sum * d + i;
            StVec<VEC> y;
#pragma unroll
            for (int e = 0; e < VEC; ++e) y.v[e] = 0.0f;
            for (int k = 0; k < a.n_sum; ++k) {
                if (k < a.n_ids && a.ids[src * a.n_ids + k] < 0) {  // (the same for the whole workgroup)
                    const float weight = a.weights[src * a.n_ids + k];
                    const T* h = static_cast<const T*>(a.h) + src * d + i;
#pragma unroll
                    for (int e = 0; e < VEC; ++e) y.v[e] = fmaf(weight, to_float<T>(h[e]), y.v[e]);
                } else {
                    const StVec<VEC> r = st_load<VEC>(yr + static_cast<int64_t>(k) * d);
#pragma unroll
                    for (int e = 0; e < VEC; ++e) y.v[e] += r.v[e];
                }
            }
            StVec<VEC> z[S];
#pragma unroll
            for (int to = 0; to < S; ++to)
#pragma unroll
                for (int e = 0; e < VEC; ++e) {
                    float v = add[to] * y.v[e];
#pragma unroll
                    for (int s = 0; s < S; ++s) v = fmaf(mix[s][to], x[s].v[e], v);
                    z[to].v[e] = v;
                }
#pragma unroll
            for (int s = 0; s < S; ++s) x[s] = z[s];
        }
        if (a.y != nullptr || a.enter != nullptr) {
#pragma unroll
            for (int s = 0; s < S; ++s) {
                if constexpr (VEC == 4) store4<float>(xr + static_cast<int64_t>(s) * d + i, x[s].v);
                else xr[static_cast<int64_t>(s) * d + i] = x[s].v[0];
            }
        }
        return read_off(x);
    };
    StVec<VEC> held[ST_HELD];
    float ss = 0.0f;
#pragma unroll
    for (int j = 0; j < ST_HELD; ++j) {
        const int g = threadIdx.x + j * ST_THREADS;
        if (g < groups) {
            held[j] = update(g * VEC);
#pragma unroll
            for (int e = 0; e < VEC; ++e) ss = fmaf(held[j].v[e], held[j].v[e], ss);
        }
    }
    for (int g = threadIdx.x + ST_HELD * ST_THREADS; g < groups; g += ST_THREADS) {
        const StVec<VEC> u = update(g * VEC);
#pragma unroll
        for (int e = 0; e < VEC; ++e) ss = fmaf(u.v[e], u.v[e], ss);
    }
    if (a.out == nullptr) return;
    ss = wave_sum(ss);
    if (threadIdx.x % kWave == 0) red[threadIdx.x / kWave] = ss;
    __syncthreads();
    float total = 0.0f;
#pragma unroll
    for (int i = 0; i < ST_THREADS / kWave; ++i) total += red[i];
    const float scale = 1.0f / sqrtf(total / static_cast<float>(d) + a.eps);
    T* o = static_cast<T*>(a.out) + static_cast<int64_t>(t) * d;
    auto finish = [&](int i, const StVec<VEC>& u) {
        float v[VEC];
#pragma unroll
        for (int e = 0; e < VEC; ++e) v[e] = u.v[e] * scale;
        if (a.w != nullptr) {
            const StVec<VEC> w = st_load<VEC>(a.w + i);
#pragma unroll
            for (int e = 0; e < VEC; ++e) v[e] *= w.v[e];
        }
        if constexpr (VEC == 4) store4<T>(o + i, v);
        else o[i] = from_float<T>(v[0]);
    };
#pragma unroll
    for (int j = 0; j < ST_HELD; ++j) {
        const int g = threadIdx.x + j * ST_THREADS;
        if (g < groups) finish(g * VEC, held[j]);
    }
    for (int g = threadIdx.x + ST_HELD * ST_THREADS; g < groups; g += ST_THREADS) {
        StVec<VEC> x[S];
#pragma unroll
        for (int s = 0; s < S; ++s) x[s] = st_load<VEC>(xr + static_cast<int64_t>(s) * d + g * VEC);  // (each thread reads what it wrote)
        finish(g * VEC, read_off(x));
    }
}

template <typename T, int VEC>
void launch_streams(const StreamsArgs& a, int n, int S, hipStream_t stream) {
    switch (S) {
        case 1: streams_update_kernel<T, 1, VEC><<<n, ST_THREADS, 0, stream>>>(a); break;
        case 2: streams_update_kernel<T, 2, VEC><<<n, ST_THREADS, 0, stream>>>(a); break;
        case 3: streams_update_kernel<T, 3, VEC><<<n, ST_THREADS, 0, stream>>>(a); break;
        case 4: streams_update_kernel<T, 4, VEC><<<n, ST_THREADS, 0, stream>>>(a); break;
        case 5: streams_update_kernel<T, 5, VEC><<<n, ST_THREADS, 0, stream>>>(a); break;
        case 6: streams_update_kernel<T, 6, VEC><<<n, ST_THREADS, 0, stream>>>(a); break;
        case 7: streams_update_kernel<T, 7, VEC><<<n, ST_THREADS, 0, stream>>>(a); break;
        default: streams_update_kernel<T, 8, VEC><<<n, ST_THREADS, 0, stream>>>(a); break;
    }
}

}  // namespace liyab

using namespace liyab;

// x: float [rows of the step, S, d]; enter: float [rows, d] or null (it may not lie in x unless S is 1 and it is x); y: float
// [rows * n_sum, d] or null; ids, weights [rows * n_ids] and h [rows, d] in out_dtype with n_ids > 0; mix: float [S, S] ([from, to]), add, in: float
// [S], w: float [d], each or null; out [n, d] in out_dtype or null; rows: int [n] or null (then nothing is written to x).
extern "C" int liyab_streams_update(float* x, const float* enter, const float* y, int n_sum, const int* ids, const float* weights, int n_ids,
                                    const void* h, const float* mix, const float* add, const float* in, const float* w, float eps, void* out,
                                    int out_dtype, const int* rows, int n, int S, int d, hipStream_t stream) {
    LIYAB_REQUIRE(x && (enter || y || out), "streams_update: null pointer");
    LIYAB_REQUIRE(n >= 0 && d > 0 && S >= 1 && S <= ST_MAX_STREAMS, "streams_update: bad sizes n=%d d=%d, %d streams (up to %d)", n, d, S, ST_MAX_STREAMS);
    LIYAB_REQUIRE(y == nullptr || n_sum >= 1, "streams_update: %d rows a token", n_sum);
    LIYAB_REQUIRE(n_ids == 0 || (y && ids && weights && h && n_ids > 0 && n_ids <= n_sum), "streams_update: identity entries need the router's lists and the rows it read");
    LIYAB_REQUIRE(rows == nullptr || (y == nullptr && enter == nullptr && out), "streams_update: gathered rows are only read");
    LIYAB_REQUIRE(out_dtype == kF32 || out_dtype == kBF16, "streams_update: unknown dtype %d", out_dtype);
    if (n == 0) return 0;
    const StreamsArgs a{x, enter, y, n_sum, n_ids, ids, weights, h, mix, add, in, w, eps, out, rows, d};
    const auto aligned = [](const void* p) { return (reinterpret_cast<uintptr_t>(p) & 15) == 0; };
    const bool vec = d % 4 == 0 && aligned(x) && aligned(enter) && aligned(y) && aligned(w) && aligned(out);
    if (out_dtype == kF32) {
        if (vec) launch_streams<float, 4>(a, n, S, stream);
        else launch_streams<float, 1>(a, n, S, stream);
    } else {
        if (vec) launch_streams<bf16_t, 4>(a, n, S, stream);
        else launch_streams<bf16_t, 1>(a, n, S, stream);
    }
    return check_launch("streams_update");
}
