// Shared by the row-by-row and the chunked kernels of the linear recurrences (not part of the C ABI).
#pragma once
#include "common.h"

constexpr int kMaxRank = 256;  // of the low-rank decay projection

__device__ __forceinline__ float silu_f32(float v) { return v / (1.0f + expf(-v)); }
__device__ __forceinline__ float sigmoid_f32(float v) { return 1.0f / (1.0f + expf(-v)); }
__device__ __forceinline__ float softplus_f32(float v) { return fmaxf(v, 0.f) + log1pf(expf(-fabsf(v))); }

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

struct RecParams {
    mi355_recurrent_args a;
    mi355_seq_batch b;
    int parts, slices;  // row kernel: row parts of the state, 64-column slices
};

// one convolution output: channel c of the q | k | v inputs (`off` = its column in proj, `cr` = its column in the ring), row i of the
// portion that starts at position pos0
template <typename T>
__device__ __forceinline__ float conv_at(const mi355_recurrent_args& a, const T* rows, const T* ring, int ring_ld, int off, int cr,
                                         const float* w, int i, int pos0) {
    float v = 0.f;
    for (int j = 0; j < a.taps; ++j) {  // j rows back
        const int r = i - j;
        float x = 0.f;
        if (r >= 0)
            x = to_f32<T>(rows[(int64_t)r * a.ld + off]);
        else if (pos0 + r >= 0)
            x = to_f32<T>(ring[(int64_t)((pos0 + r) % a.taps) * ring_ld + cr]);
        v += w[a.taps - 1 - j] * x;
    }
    return silu_f32(v);
}

// recurrent_chunks.hip
bool mi355_recurrent_chunks_fit(const mi355_recurrent_args& a, const mi355_seq_batch& b);
int mi355_recurrent_chunks(const RecParams& r, hipStream_t s);
