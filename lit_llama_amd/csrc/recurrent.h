// Shared by the row-by-row and the chunked kernels of the linear recurrences (not part of the C ABI).
#pragma once
#include <type_traits>

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

// where input row r of a portion lies (rows of earlier portions below 0: in the ring).  Always a readable address, `ok` = the row exists:
// loads without branches, so that all of a thread's requests are in flight together
template <typename T>
__device__ __forceinline__ const T* conv_input(const mi355_recurrent_args& a, const T* rows, const T* ring, int ring_ld, int off, int cr, int r,
                                               int pos0, bool& ok) {
    ok = ok && pos0 + r >= 0;
    const T* old = ring + (int64_t)((unsigned)(ok ? pos0 + r : 0) % (unsigned)a.taps) * ring_ld + cr;
    return r >= 0 ? rows + (int64_t)r * a.ld + off : old;
}

// one convolution output: channel c of the q | k | v inputs (`off` = its column in proj, `cr` = its column in the ring), row i of the
// portion that starts at position pos0
template <typename T>
__device__ __forceinline__ float conv_at(const mi355_recurrent_args& a, const T* rows, const T* ring, int ring_ld, int off, int cr,
                                         const float* w, int i, int pos0, float bias = 0.f) {
    float v = bias;
    for (int j0 = 0; j0 < a.taps; j0 += 4) {
        T x[4];
        float wj[4];
        bool ok[4];
#pragma unroll
        for (int j = 0; j < 4; ++j) {
            ok[j] = j0 + j < a.taps;
            const int back = ok[j] ? j0 + j : 0;
            x[j] = *conv_input<T>(a, rows, ring, ring_ld, off, cr, i - back, pos0, ok[j]);
            wj[j] = w[a.taps - 1 - back];
        }
#pragma unroll
        for (int j = 0; j < 4; ++j) v += ok[j] ? wj[j] * to_f32<T>(x[j]) : 0.f;
    }
    return silu_f32(v);
}

// the same for 16 rows i .. i + 15 of one channel (rows past n give 0)
template <typename T>
__device__ __forceinline__ void conv_rows16(const mi355_recurrent_args& a, const T* rows, const T* ring, int ring_ld, int off, int cr,
                                            const float* w, int i, int n, int pos0, float (&out)[16], float bias = 0.f) {
    if (a.taps > kTaps) {
#pragma unroll
        for (int t = 0; t < 16; ++t) out[t] = i + t < n ? conv_at<T>(a, rows, ring, ring_ld, off, cr, w, i + t, pos0, bias) : 0.f;
        return;
    }
    T raw[16 + kTaps - 1];
    float x[16 + kTaps - 1], wj[kTaps];
    bool ok[16 + kTaps - 1];
#pragma unroll
    for (int e = 0; e < 16 + kTaps - 1; ++e) {
        const int r = i + e - (kTaps - 1);
        ok[e] = e > kTaps - 1 - a.taps && r < n;
        raw[e] = *conv_input<T>(a, rows, ring, ring_ld, off, cr, ok[e] ? r : 0, pos0, ok[e]);
    }
#pragma unroll
    for (int j = 0; j < kTaps; ++j) wj[j] = w[j < a.taps ? a.taps - 1 - j : 0];
#pragma unroll
    for (int e = 0; e < 16 + kTaps - 1; ++e) x[e] = ok[e] ? to_f32<T>(raw[e]) : 0.f;
#pragma unroll
    for (int j = 0; j < kTaps; ++j) wj[j] = j < a.taps ? wj[j] : 0.f;
#pragma unroll
    for (int t = 0; t < 16; ++t) {
        float v = bias;
#pragma unroll
        for (int j = 0; j < kTaps; ++j) v += wj[j] * x[kTaps - 1 + t - j];
        out[t] = i + t < n ? silu_f32(v) : 0.f;
    }
}

// log of a WKV key channel's decay, exp(-exp(z)): below -104 the decay is 0 in f32, and sums of many stay finite
__device__ __forceinline__ float wkv_log_decay(float z) { return fmaxf(-expf(z), -104.f); }

// kinds with short convolutions on q, k and v
__host__ __device__ constexpr bool has_conv(int kind) { return kind == MI355_REC_DELTA || kind == MI355_REC_SSD; }
// bias of convolution channel c
__device__ __forceinline__ float conv_bias(const float* b, int c) { return b != nullptr ? b[c] : 0.f; }
// how a kind stores its outputs
template <int KIND, typename T>
using out_t = std::conditional_t<KIND == MI355_REC_SSD, float, T>;

struct RecParams {
    mi355_recurrent_args a;
    mi355_seq_batch b;
    int parts, slices;  // row kernel: row parts of the state, 64-column slices
};

// recurrent_chunks.hip
bool mi355_recurrent_chunks_fit(const mi355_recurrent_args& a, const mi355_seq_batch& b);
int mi355_recurrent_chunks(const RecParams& r, hipStream_t s);
