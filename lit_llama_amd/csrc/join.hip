// What stands between two sublayers whose result is normalised before it joins the stream (mi355_join_rows): gate, norm of the result, residual sum,
// weighted average over the stream's earlier values, and the norm of what the next sublayer reads, in one pass over every row.  Everything is f32
// but the operands that are stored for a product.
#include "common.h"

namespace {

constexpr int kThreads = 512;

// e^v by the hardware's 2^x: sigmoid(v) within a few roundings
__device__ __forceinline__ float sigmoid_fast(float v) { return __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(v * -1.44269504088896340736f)); }
__device__ __forceinline__ float square_sum(f32x4 v) { return (v[0] * v[0] + v[1] * v[1]) + (v[2] * v[2] + v[3] * v[3]); }

// sum over the workgroup (DPP steps and one LDS pass); `red`: 8 floats that nobody else uses
__device__ __forceinline__ float sum_all(float v, float* red) {
    v = group_sum(v, 64);
    if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = v;
    __syncthreads();
    float s = 0.f;
    for (int w = 0; w < (int)(blockDim.x >> 6); ++w) s += red[w];
    return s;
}

// One row per workgroup, four consecutive values per thread, H times; the row stays in registers
template <typename T, int H>
__global__ __launch_bounds__(kThreads) void join_kernel(const mi355_join_args p) {
    __shared__ float red[2][kThreads / 64];
    const int m = blockIdx.x, nt = blockDim.x, W = p.width;
    const T* emb = p.embed != nullptr ? (const T*)p.embed + (int64_t)min(max(p.tokens[m], 0), p.vocab - 1) * W : nullptr;
    const f32x4 zero = {0.f, 0.f, 0.f, 0.f};
    f32x4 u[H], x[H], g[H], post[H], next[H], before[H];
    auto at = [&](int i) { return 4 * ((int)threadIdx.x + nt * i); };
    // (every request of the row in front of the first sum)
#pragma unroll
    for (int i = 0; i < H; ++i) {
        const int k = at(i);
        const bool in = k < W;
        u[i] = !in ? zero : emb != nullptr ? get4(emb + k) : *(const f32x4*)(p.t + (int64_t)m * p.ldt + k);
        x[i] = in && emb == nullptr ? *(const f32x4*)(p.x + (int64_t)m * p.ldx + k) : zero;
        g[i] = zero;
        if (in && p.gate != nullptr)
            g[i] = p.gate_dtype == MI355_F32 ? *(const f32x4*)((const float*)p.gate + (int64_t)m * p.ld_gate + k)
                                             : get4((const bf16_t*)p.gate + (int64_t)m * p.ld_gate + k);
        post[i] = in && p.post != nullptr ? get4((const T*)p.post + k) + p.norm_add : zero;
        next[i] = in && p.next != nullptr ? get4((const T*)p.next + k) + p.norm_add : zero;
    }
#pragma unroll
    for (int i = 0; i < H; ++i) before[i] = zero;
#pragma unroll(H > 2 ? 2 : 4)
    for (int j = 0; j < p.n_stream; ++j) {
        const float w = p.average[j];
        const float* row = p.stream + j * p.stream_stride + (int64_t)m * p.ldx;
#pragma unroll
        for (int i = 0; i < H; ++i) before[i] += w * (at(i) < W ? *(const f32x4*)(row + at(i)) : zero);
    }
    if (p.gate != nullptr) {
#pragma unroll
        for (int i = 0; i < H; ++i)
#pragma unroll
            for (int e = 0; e < 4; ++e) u[i][e] *= sigmoid_fast(g[i][e]);
    }
    if (p.post != nullptr) {
        float ss = 0.f;
#pragma unroll
        for (int i = 0; i < H; ++i) ss += square_sum(u[i]);
        const float r = 1.0f / sqrtf(sum_all(ss, red[0]) / (float)W + p.eps);
#pragma unroll
        for (int i = 0; i < H; ++i) u[i] = u[i] * r * post[i];
    }
#pragma unroll
    for (int i = 0; i < H; ++i) x[i] += u[i];
    if (p.stream_out != nullptr) {
#pragma unroll
        for (int i = 0; i < H; ++i)
            if (at(i) < W) *(f32x4*)(p.stream_out + (int64_t)m * p.ldx + at(i)) = x[i];
    }
    if (p.n_stream > 0) {
        const float own = p.average[p.n_stream];
#pragma unroll
        for (int i = 0; i < H; ++i) x[i] = before[i] + own * x[i];
    }
#pragma unroll
    for (int i = 0; i < H; ++i)
        if (at(i) < W) *(f32x4*)(p.x + (int64_t)m * p.ldx + at(i)) = x[i];
    if (p.next != nullptr) {
        float ss = 0.f;
#pragma unroll
        for (int i = 0; i < H; ++i) ss += at(i) < W ? square_sum(x[i]) : 0.f;
        const float r = 1.0f / sqrtf(sum_all(ss, red[1]) / (float)W + p.eps);
#pragma unroll
        for (int i = 0; i < H; ++i)
            if (at(i) < W) put4((T*)p.h + (int64_t)m * p.ldh + at(i), x[i] * r * next[i]);
    }
}

// any width: a value at a time; what a thread writes to x it alone reads again
template <typename T>
__global__ __launch_bounds__(kThreads) void join_any_kernel(const mi355_join_args p) {
    __shared__ float red[32];
    constexpr int kType = sizeof(T) == 4 ? MI355_F32 : MI355_BF16;
    const int m = blockIdx.x, W = p.width;
    const int64_t emb = p.embed != nullptr ? (int64_t)min(max(p.tokens[m], 0), p.vocab - 1) * W : 0;
    float* x = p.x + (int64_t)m * p.ldx;
    auto result = [&](int k) {
        float u = p.embed != nullptr ? ld_as_f32(p.embed, emb + k, kType) : p.t[(int64_t)m * p.ldt + k];
        if (p.gate != nullptr) u *= sigmoid_fast(ld_as_f32(p.gate, (int64_t)m * p.ld_gate + k, p.gate_dtype));
        return u;
    };
    float r = 1.f;
    if (p.post != nullptr) {
        float ss = 0.f;
        for (int k = threadIdx.x; k < W; k += kThreads) ss += result(k) * result(k);
        r = 1.0f / sqrtf(block_sum(ss, red) / (float)W + p.eps);
    }
    float ss = 0.f;
    for (int k = threadIdx.x; k < W; k += kThreads) {
        float v = result(k);
        if (p.post != nullptr) v = v * r * (ld_as_f32(p.post, k, kType) + p.norm_add);
        if (p.embed == nullptr) v += x[k];
        if (p.stream_out != nullptr) p.stream_out[(int64_t)m * p.ldx + k] = v;
        if (p.n_stream > 0) {
            v *= p.average[p.n_stream];
            for (int j = 0; j < p.n_stream; ++j) v += p.average[j] * p.stream[j * p.stream_stride + (int64_t)m * p.ldx + k];
        }
        x[k] = v;
        ss += v * v;
    }
    if (p.next != nullptr) {
        const float rn = 1.0f / sqrtf(block_sum(ss, red) / (float)W + p.eps);
        for (int k = threadIdx.x; k < W; k += kThreads)
            st_from_f32(p.h, (int64_t)m * p.ldh + k, kType, x[k] * rn * (ld_as_f32(p.next, k, kType) + p.norm_add));
    }
}

template <typename T>
int launch(const mi355_join_args& a, hipStream_t s) {
    const int size = dtype_size(a.gate_dtype);
    const bool vec = a.width % 4 == 0 && a.width <= 16 * kThreads && a.ldx % 4 == 0 && a.ldh % 4 == 0 && a.ldt % 4 == 0 && a.ld_gate % 4 == 0 &&
                     (uintptr_t)a.x % 16 == 0 && (uintptr_t)a.t % 16 == 0 && (uintptr_t)a.gate % (4 * size) == 0 && (uintptr_t)a.h % 16 == 0 &&
                     (uintptr_t)a.post % 16 == 0 && (uintptr_t)a.next % 16 == 0 && (uintptr_t)a.embed % 16 == 0 && (uintptr_t)a.stream % 16 == 0 &&
                     (uintptr_t)a.stream_out % 16 == 0 && a.stream_stride % 4 == 0;
    if (!vec) hipLaunchKernelGGL(join_any_kernel<T>, dim3(a.rows), dim3(kThreads), 0, s, a);
    else if (a.width <= 1024) hipLaunchKernelGGL((join_kernel<T, 1>), dim3(a.rows), dim3(256), 0, s, a);
    else if (a.width <= 2048) hipLaunchKernelGGL((join_kernel<T, 1>), dim3(a.rows), dim3(512), 0, s, a);
    else if (a.width <= 4096) hipLaunchKernelGGL((join_kernel<T, 2>), dim3(a.rows), dim3(512), 0, s, a);
    else hipLaunchKernelGGL((join_kernel<T, 4>), dim3(a.rows), dim3(512), 0, s, a);
    MI355_LAUNCH_CHECK();
    return 0;
}

}  // namespace

extern "C" int mi355_join_rows(const mi355_join_args* a, mi355_stream_t stream) {
    MI355_CHECK_ARG(a && a->x && (a->embed ? a->tokens != nullptr && a->vocab > 0 : a->t != nullptr), MI355_E_ARG, "join_rows: null argument");
    MI355_CHECK_ARG(a->dtype == MI355_F32 || a->dtype == MI355_BF16, MI355_E_DTYPE, "join_rows: dtype must be f32 or bf16");
    MI355_CHECK_ARG(a->gate == nullptr || a->gate_dtype == MI355_F32 || a->gate_dtype == MI355_BF16, MI355_E_DTYPE, "join_rows: a gate is f32 or bf16");
    MI355_CHECK_ARG(a->rows > 0 && a->width > 0 && a->ldx >= a->width && (a->embed || a->ldt >= a->width) && (a->gate == nullptr || a->ld_gate >= a->width) &&
                        (a->next == nullptr || (a->h && a->ldh >= a->width)),
                    MI355_E_SHAPE, "join_rows: %d rows of %d do not fit their pitches", a->rows, a->width);
    MI355_CHECK_ARG(a->n_stream >= 0 && (a->n_stream == 0 || (a->stream && a->average && a->stream_stride >= (int64_t)(a->rows - 1) * a->ldx + a->width)),
                    MI355_E_ARG, "join_rows: bad stream");
    return a->dtype == MI355_F32 ? launch<float>(*a, (hipStream_t)stream) : launch<bf16_t>(*a, (hipStream_t)stream);
}
