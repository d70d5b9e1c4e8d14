// Shared by the row-by-row and the chunked kernels of the linear recurrences (not part of the C ABI).
#pragma once
#include "common.h"

constexpr int kMaxRank = 256;  // of the low-rank decay projection

// e^v by the hardware's 2^x: one rounding of v log2(e) (relative error |v| 2^-24) and v_exp_f32's own
__device__ __forceinline__ float exp_f32(float v) { return __builtin_amdgcn_exp2f(v * 1.44269504088896340736f); }
__device__ __forceinline__ float sigmoid_f32(float v) { return __builtin_amdgcn_rcpf(1.0f + exp_f32(-v)); }
__device__ __forceinline__ float silu_f32(float v) { return v * sigmoid_f32(v); }
// log(1 + u) for u in [0, 1]: log(w) u / (w - 1) with w = 1 + u rounded, whose error cancels in the quotient (Goldberg, "What Every Computer
// Scientist Should Know About Floating-Point Arithmetic", 1991, theorem 4)
__device__ __forceinline__ float log1p_unit(float u) {
    const float w = 1.0f + u, d = w - 1.0f;
    return d == 0.f ? u : __builtin_amdgcn_logf(w) * 0.69314718055994530942f * u * __builtin_amdgcn_rcpf(d);
}
__device__ __forceinline__ float softplus_f32(float v) { return fmaxf(v, 0.f) + log1p_unit(exp_f32(-fabsf(v))); }

template <typename T>
__device__ __forceinline__ float to_f32(T v);
template <>
__device__ __forceinline__ float to_f32<float>(float v) { return v; }
template <>
__device__ __forceinline__ float to_f32<bf16_t>(bf16_t v) { return bf16_to_f32(v); }
template <typename T>
__device__ __forceinline__ T from_f32(float v);
template <>
__device__ __forceinline__ float from_f32<float>(float v) { return v; }
template <>
__device__ __forceinline__ bf16_t from_f32<bf16_t>(float v) { return f32_to_bf16(v); }

constexpr int kTaps = 8;  // taps a thread keeps in registers; longer convolutions take the loops

// one convolution output: channel c of the q | k | v inputs (`off` = its column in proj, `cr` = its column in the ring), row i of the
// portion that starts at position pos0
template <typename T>
__device__ __forceinline__ float conv_at(const mi355_recurrent_args& a, const T* rows, const T* ring, int ring_ld, int off, int cr,
                                         const float* w, int i, int pos0) {
    auto input = [&](int r) {  // row r of the portion, rows of earlier portions below 0
        if (r >= 0) return to_f32<T>(rows[(int64_t)r * a.ld + off]);
        return pos0 + r >= 0 ? to_f32<T>(ring[(int64_t)((pos0 + r) % a.taps) * ring_ld + cr]) : 0.f;
    };
    float v = 0.f;
    if (a.taps <= kTaps) {
        float x[kTaps], wj[kTaps];
#pragma unroll
        for (int j = 0; j < kTaps; ++j) {
            x[j] = j < a.taps ? input(i - j) : 0.f;
            wj[j] = j < a.taps ? w[a.taps - 1 - j] : 0.f;
        }
#pragma unroll
        for (int j = 0; j < kTaps; ++j) v += wj[j] * x[j];
    } else {
        for (int j = 0; j < a.taps; ++j) v += w[a.taps - 1 - j] * input(i - j);
    }
    return silu_f32(v);
}

// the same for 16 rows i .. i + 15 of one channel (rows past n give 0)
template <typename T>
__device__ __forceinline__ void conv_rows16(const mi355_recurrent_args& a, const T* rows, const T* ring, int ring_ld, int off, int cr,
                                            const float* w, int i, int n, int pos0, float (&out)[16]) {
    if (a.taps > kTaps) {
#pragma unroll
        for (int t = 0; t < 16; ++t) out[t] = i + t < n ? conv_at<T>(a, rows, ring, ring_ld, off, cr, w, i + t, pos0) : 0.f;
        return;
    }
    float x[16 + kTaps - 1], wj[kTaps];
#pragma unroll
    for (int e = 0; e < 16 + kTaps - 1; ++e) {
        const int r = i + e - (kTaps - 1);
        x[e] = 0.f;
        if (e > kTaps - 1 - a.taps && r < n) {
            if (r >= 0)
                x[e] = to_f32<T>(rows[(int64_t)r * a.ld + off]);
            else if (pos0 + r >= 0)
                x[e] = to_f32<T>(ring[(int64_t)((pos0 + r) % a.taps) * ring_ld + cr]);
        }
    }
#pragma unroll
    for (int j = 0; j < kTaps; ++j) wj[j] = j < a.taps ? w[a.taps - 1 - j] : 0.f;
#pragma unroll
    for (int t = 0; t < 16; ++t) {
        float v = 0.f;
#pragma unroll
        for (int j = 0; j < kTaps; ++j) v += wj[j] * x[kTaps - 1 + t - j];
        out[t] = i + t < n ? silu_f32(v) : 0.f;
    }
}

struct RecParams {
    mi355_recurrent_args a;
    mi355_seq_batch b;
    int parts, slices;  // row kernel: row parts of the state, 64-column slices
};

// recurrent_chunks.hip
bool mi355_recurrent_chunks_fit(const mi355_recurrent_args& a, const mi355_seq_batch& b);
int mi355_recurrent_chunks(const RecParams& r, hipStream_t s);
