// The forward pass of a layered hybrid model (mi355_hybrid_forward): a host-side walk over the layer runs that enqueues this library's
// linears (gemv.hip for a few rows, gemm.hip above, the exact f32 kernel for f32 models), mixers (window_attention.hip, recurrent.hip) and
// experts (experts.hip).  RMSNorm rides in the consuming linear and the residual sum in the producing one; the residual stream is f32.
// A parallel layer normalises its row once (by groups, with the token shift of its mixer), and its mixer's output and hidden row leave
// through one product.  A sandwich layer's sublayers read rows that the pass behind the sublayer in front (join.hip) has normalised.
#include "product.h"

namespace {

// one row per workgroup; columns width .. ldx - 1 are zero
__global__ __launch_bounds__(256) void embed_rows_kernel(const int32_t* tokens, const void* wte, int dtype, float* x, int width, int ldx,
                                                         int vocab) {
    const int m = blockIdx.x;
    const int tok = min(max(tokens[m], 0), vocab - 1);
    float* dst = x + (int64_t)m * ldx;
    if (dtype == MI355_BF16 && width % 8 == 0) {  // (ldx is a multiple of 16)
        const u32x4* src = (const u32x4*)((const bf16_t*)wte + (int64_t)tok * width);
        for (int j = threadIdx.x; j < ldx / 8; j += 256) {
            const u32x4 r = j < width / 8 ? src[j] : u32x4{0u, 0u, 0u, 0u};
            f32x4 lo, hi;
#pragma unroll
            for (int e = 0; e < 2; ++e) {
                lo[2 * e] = __uint_as_float(r[e] << 16), lo[2 * e + 1] = __uint_as_float(r[e] & 0xffff0000u);
                hi[2 * e] = __uint_as_float(r[2 + e] << 16), hi[2 * e + 1] = __uint_as_float(r[2 + e] & 0xffff0000u);
            }
            ((f32x4*)dst)[2 * j] = lo;
            ((f32x4*)dst)[2 * j + 1] = hi;
        }
        return;
    }
    for (int k = threadIdx.x; k < ldx; k += 256) dst[k] = k < width ? ld_as_f32(wte, (int64_t)tok * width + k, dtype) : 0.f;
}

__global__ __launch_bounds__(256) void gather_rows_kernel(const float* x, const int32_t* want, float* xw, int ldx) {
    const int64_t src = (int64_t)want[blockIdx.x] * ldx, dst = (int64_t)blockIdx.x * ldx;
    for (int k = threadIdx.x; k < ldx; k += 256) xw[dst + k] = x[src + k];
}

// xb[m] = bf16(norm(x[m]) * scale), one row per workgroup: the operand of a wide product, multiplied where it lies.  K % 128 == 0, so rows
// are whole 16-B vectors
__global__ __launch_bounds__(512) void norm_rows_kernel(const float* x, int64_t ldx, const void* scale, int scale_dtype, float eps, int K,
                                                        float norm_add, bf16_t* xb) {
    __shared__ float red[32];
    const f32x4* row = (const f32x4*)(x + (int64_t)blockIdx.x * ldx);
    constexpr int kHeld = 4;  // vectors a thread keeps between the two passes
    f32x4 v[kHeld];
    float ss = 0.f;
#pragma unroll
    for (int i = 0; i < kHeld; ++i) {
        const int j = threadIdx.x + i * 512;
        v[i] = j < K / 4 ? row[j] : f32x4{0.f, 0.f, 0.f, 0.f};
        ss += (v[i][0] * v[i][0] + v[i][1] * v[i][1]) + (v[i][2] * v[i][2] + v[i][3] * v[i][3]);
    }
    for (int j = threadIdx.x + kHeld * 512; j < K / 4; j += 512) {
        const f32x4 w = row[j];
        ss += (w[0] * w[0] + w[1] * w[1]) + (w[2] * w[2] + w[3] * w[3]);
    }
    const float rinv = 1.0f / sqrtf(block_sum(ss, red) / (float)K + eps);
    u32x2* out = (u32x2*)(xb + (int64_t)blockIdx.x * K);
    typedef __attribute__((ext_vector_type(2))) __bf16 bf2;
    auto put = [&](int j, f32x4 w) {
        float s[4];
        if (scale_dtype == MI355_BF16) {
            const u32x2 r = ((const u32x2*)scale)[j];
            s[0] = __uint_as_float(r[0] << 16), s[1] = __uint_as_float(r[0] & 0xffff0000u);
            s[2] = __uint_as_float(r[1] << 16), s[3] = __uint_as_float(r[1] & 0xffff0000u);
        } else {
            for (int e = 0; e < 4; ++e) s[e] = ld_as_f32(scale, 4 * j + e, scale_dtype);
        }
        for (int e = 0; e < 4; ++e) s[e] += norm_add;
        const bf2 a = {(__bf16)(w[0] * rinv * s[0]), (__bf16)(w[1] * rinv * s[1])}, b = {(__bf16)(w[2] * rinv * s[2]), (__bf16)(w[3] * rinv * s[3])};
        out[j] = u32x2{__builtin_bit_cast(uint32_t, a), __builtin_bit_cast(uint32_t, b)};
    };
#pragma unroll
    for (int i = 0; i < kHeld; ++i) {
        const int j = threadIdx.x + i * 512;
        if (j < K / 4) put(j, v[i]);
    }
    for (int j = threadIdx.x + kHeld * 512; j < K / 4; j += 512) put(j, row[j]);
}

// ---- parallel layers: h = norm(x) in groups, and the mixes h + (h' - h) mu of the token shift (h' = the row before)
struct NormParams : mi355_norm_args {
    int size;               // of a group
    mi355_seq_batch b;
};

// One row per workgroup.  H > 0: rows of up to 2048 H values whose groups are whole runs of 256 (a wave's load), held in registers; H = 0: any
// width, and with MIX a second row: the row before, or, in the workgroup of a portion's first row, the portion's last one (it enters the
// state there).  Dynamic LDS: sums of squares [2][max(runs, 8, groups)], 1 / rms [2][groups]
template <typename T, bool MIX, int H>
__global__ __launch_bounds__(512) void norm_groups_kernel(const NormParams p) {
    static_assert(!MIX || H == 0, "rows with mixes in registers: norm_mix_kernel");
    extern __shared__ __attribute__((aligned(16))) float sm[];
    __shared__ int s_seq;
    const int m = blockIdx.x, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const int per = H > 0 ? p.size / 256 : p.groups < 8 ? 8 / p.groups : 1;  // sums per group
    const int n_sums = p.groups * per;
    float* sums = sm;                     // [2][n_sums]
    float* rinv = sm + 2 * n_sums;        // [2][groups]
    const float* row = p.x + (int64_t)(p.want != nullptr ? p.want[m] : m) * p.ldx;
    const float* other = row;
    int seq = 0, i = 0;
    if constexpr (MIX) {
        seq = m;
        if (p.b.max_count > 1) {
            for (int s = tid; s < p.b.seqs; s += 512)
                if (m >= p.b.row0[s] && m < p.b.row0[s] + p.b.count[s]) s_seq = s;
            __syncthreads();
            seq = s_seq;
            i = m - p.b.row0[seq];
            other = i > 0 ? row - p.ldx : row + (int64_t)(p.b.count[seq] - 1) * p.ldx;
        }
    }
    constexpr int HH = H > 0 ? H : 1;
    f32x4 a[HH], sc[HH];
    if constexpr (H > 0) {
#pragma unroll
        for (int j = 0; j < H; ++j) {
            const int k = 4 * (tid + 512 * j);
            a[j] = k < p.width ? *(const f32x4*)(row + k) : f32x4{0.f, 0.f, 0.f, 0.f};
        }
#pragma unroll
        for (int j = 0; j < H; ++j) {
            const int k = 4 * (tid + 512 * j);
            sc[j] = k < p.width ? get4((const T*)p.scale + k) : f32x4{0.f, 0.f, 0.f, 0.f};
        }
#pragma unroll
        for (int j = 0; j < H; ++j) {
            const float s0 = group_sum((a[j][0] * a[j][0] + a[j][1] * a[j][1]) + (a[j][2] * a[j][2] + a[j][3] * a[j][3]), 64);
            if (lane == 0 && wave + 8 * j < n_sums) sums[wave + 8 * j] = s0;
        }
    } else {
        const int seg = (p.size + per - 1) / per;
        for (int q = wave; q < n_sums; q += 8) {
            const int gr = q / per, v0 = (q - gr * per) * seg, v1 = min(p.size, v0 + seg);
            const int64_t at = (int64_t)gr * p.size;
            float s0 = 0.f, s1 = 0.f;
            for (int v = v0 + lane; v < v1; v += 64) {
                s0 += row[at + v] * row[at + v];
                if constexpr (MIX) s1 += other[at + v] * other[at + v];
            }
            s0 = group_sum(s0, 64);
            s1 = group_sum(s1, 64);
            if (lane == 0) {
                sums[q] = s0;
                if constexpr (MIX) sums[n_sums + q] = s1;
            }
        }
    }
    __syncthreads();
    for (int q = tid; q < (MIX ? 2 : 1) * p.groups; q += 512) {
        float s = 0.f;
        for (int j = 0; j < per; ++j) s += sums[q * per + j];
        rinv[q] = 1.0f / sqrtf(s / (float)p.size + p.eps);
    }
    __syncthreads();
    T* h = (T*)p.h + (int64_t)m * p.ldh;
    if constexpr (H > 0) {
#pragma unroll
        for (int j = 0; j < H; ++j) {
            const int k = 4 * (tid + 512 * j);
            if (k < p.width) put4(h + k, a[j] * rinv[(wave + 8 * j) / per] * sc[j]);
        }
    } else {
        float* state = MIX ? p.shift + (int64_t)p.b.slot[seq] * p.width : nullptr;
        const bool first = MIX && i == 0, begun = first && p.b.pos[seq] > 0;
        for (int k = tid; k < p.width; k += 512) {
            const int gr = k / p.size;
            const float scale = ld_as_f32(p.scale, k, sizeof(T) == 4 ? MI355_F32 : MI355_BF16);
            const float v = row[k] * rinv[gr] * scale;
            st_from_f32(h, k, sizeof(T) == 4 ? MI355_F32 : MI355_BF16, v);
            if constexpr (MIX) {
                float d = other[k] * rinv[p.groups + gr] * scale;
                if (first) {  // (d: the portion's last row; of one row, itself)
                    const float old = begun ? state[k] : 0.f;
                    state[k] = d;
                    d = old;
                }
                d -= v;
                for (int s = 0; s < p.n_mix; ++s)
                    st_from_f32((T*)p.mix + s * p.mix_stride + (int64_t)m * p.ldh, k, sizeof(T) == 4 ? MI355_F32 : MI355_BF16,
                                v + d * p.mu[(int64_t)s * p.width + k]);
            }
        }
    }
}

// The same with the mixes, for rows of up to 2048 H values, `per_wg` consecutive rows per workgroup: the factors stay in registers, and a row is
// the next one's predecessor.  Dynamic LDS: sums of squares [2 (turns)][width / 256], 1 / rms [2][groups]
constexpr int kMixRows = 4;
template <typename T, int H>
__global__ __launch_bounds__(512) void norm_mix_kernel(const NormParams p, int rows, int per_wg) {
    extern __shared__ __attribute__((aligned(16))) float sm[];
    __shared__ int s_seq[kMixRows];
    const int m0 = blockIdx.x * per_wg, n = min(per_wg, rows - m0), tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const int per = p.size / 256, n_sums = p.groups * per;
    int turn = 0;
    f32x4 sc[H], mu[5][H], raw[H], h[H], before[H];
    auto request = [&](const float* row) {
#pragma unroll
        for (int j = 0; j < H; ++j) {
            const int k = 4 * (tid + 512 * j);
            raw[j] = k < p.width ? *(const f32x4*)(row + k) : f32x4{0.f, 0.f, 0.f, 0.f};
        }
    };
    // raw -> out = norm(raw)
    auto norm = [&](f32x4 (&out)[H]) {
        float* sums = sm + turn * n_sums;
        float* rinv = sm + 2 * n_sums + turn * p.groups;
        turn ^= 1;
#pragma unroll
        for (int j = 0; j < H; ++j) {
            out[j] = raw[j] * sc[j];
            const float s = group_sum((raw[j][0] * raw[j][0] + raw[j][1] * raw[j][1]) + (raw[j][2] * raw[j][2] + raw[j][3] * raw[j][3]), 64);
            if (lane == 0 && wave + 8 * j < n_sums) sums[wave + 8 * j] = s;
        }
        __syncthreads();
        for (int q = tid; q < p.groups; q += 512) {
            float s = 0.f;
            for (int j = 0; j < per; ++j) s += sums[q * per + j];
            rinv[q] = 1.0f / sqrtf(s / (float)p.size + p.eps);
        }
        __syncthreads();
#pragma unroll
        for (int j = 0; j < H; ++j)
            if (4 * (tid + 512 * j) < p.width) out[j] *= rinv[(wave + 8 * j) / per];
    };
    const float* row = p.x + (int64_t)m0 * p.ldx;
    request(m0 > 0 ? row - p.ldx : row);  // (the row before, in case it belongs to the same portion)
#pragma unroll
    for (int j = 0; j < H; ++j) {
        const int k = 4 * (tid + 512 * j);
        const bool in = k < p.width;
        sc[j] = in ? get4((const T*)p.scale + k) : f32x4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int s = 0; s < 5; ++s) mu[s][j] = in && s < p.n_mix ? *(const f32x4*)(p.mu + (int64_t)s * p.width + k) : f32x4{0.f, 0.f, 0.f, 0.f};
    }
    if (p.b.max_count == 1) {
        if (tid < n) s_seq[tid] = m0 + tid;
    } else {
        for (int s = tid; s < p.b.seqs; s += 512) {
            const int r0 = p.b.row0[s], r1 = r0 + p.b.count[s];
            for (int m = max(r0, m0); m < min(r1, m0 + n); ++m) s_seq[m - m0] = s;
        }
    }
    __syncthreads();
    if (p.b.row0[s_seq[0]] < m0) norm(before);
    request(row);
    for (int r = 0; r < n; ++r) {
        const int seq = s_seq[r], i = m0 + r - p.b.row0[seq], cnt = p.b.count[seq];
        norm(h);
        if (i == 0) {  // what the state holds is this row's predecessor; the portion's last row replaces it
            float* state = p.shift + (int64_t)p.b.slot[seq] * p.width;
            const bool begun = p.b.pos[seq] > 0;
            f32x4 last[H];
            if (cnt > 1) {
                request(row + (int64_t)(r + cnt - 1) * p.ldx);
                norm(last);
            }
#pragma unroll
            for (int j = 0; j < H; ++j) {
                const int k = 4 * (tid + 512 * j);
                if (k >= p.width) continue;
                before[j] = begun ? *(const f32x4*)(state + k) : f32x4{0.f, 0.f, 0.f, 0.f};
                *(f32x4*)(state + k) = cnt > 1 ? last[j] : h[j];
            }
        }
        if (r + 1 < n) request(row + (int64_t)(r + 1) * p.ldx);
        const int64_t at = (int64_t)(m0 + r) * p.ldh;
#pragma unroll
        for (int j = 0; j < H; ++j) {
            const int k = 4 * (tid + 512 * j);
            if (k >= p.width) continue;
            put4((T*)p.h + at + k, h[j]);
            const f32x4 d = before[j] - h[j];
#pragma unroll
            for (int s = 0; s < 5; ++s)
                if (s < p.n_mix) put4((T*)p.mix + s * p.mix_stride + at + k, h[j] + d * mu[s][j]);
            before[j] = h[j];
        }
    }
}

template <typename T, bool MIX>
void launch_norm(const NormParams& p, int rows, hipStream_t s) {
    const bool whole = p.size % 256 == 0 && p.width <= 8192;
    const int sums = whole ? p.width / 256 : p.groups < 8 ? 8 : p.groups;
    const size_t lds = (size_t)2 * (sums + p.groups) * 4;
    if constexpr (MIX) {
        if (whole) {
            const int per_wg = p.b.max_count == 1 ? 1 : kMixRows;
            if (p.width <= 4096) hipLaunchKernelGGL((norm_mix_kernel<T, 2>), dim3((rows + per_wg - 1) / per_wg), dim3(512), lds, s, p, rows, per_wg);
            else hipLaunchKernelGGL((norm_mix_kernel<T, 4>), dim3((rows + per_wg - 1) / per_wg), dim3(512), lds, s, p, rows, per_wg);
            return;
        }
    }
    if constexpr (!MIX) {
        if (whole) {
            if (p.width <= 4096) hipLaunchKernelGGL((norm_groups_kernel<T, false, 2>), dim3(rows), dim3(512), lds, s, p);
            else hipLaunchKernelGGL((norm_groups_kernel<T, false, 4>), dim3(rows), dim3(512), lds, s, p);
            return;
        }
    }
    hipLaunchKernelGGL((norm_groups_kernel<T, MIX, 0>), dim3(rows), dim3(512), lds, s, p);
}

// rows [gate | up] of 2 n values -> the clamped gated unit
__global__ __launch_bounds__(256) void clampglu_kernel(const float* gu, float* h, int n, int64_t ldh, int64_t total, float limit) {
    for (int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x; i < total; i += (int64_t)gridDim.x * 256) {
        const int64_t m = i / n, k = i - m * n;
        h[m * ldh + k] = clampglu_f32(gu[m * 2 * n + k], gu[m * 2 * n + n + k], limit);
    }
}

__global__ __launch_bounds__(256) void relu2_kernel(float* h, int64_t n) {
    for (int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x; i < n; i += (int64_t)gridDim.x * 256) h[i] = relu2_f32(h[i]);
}

// rows [gate | up] of 2 n values -> gelu_tanh(gate) * up
__global__ __launch_bounds__(256) void geglu_kernel(const float* gu, float* h, int n, int64_t total) {
    for (int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x; i < total; i += (int64_t)gridDim.x * 256) {
        const int64_t m = i / n, k = i - m * n;
        h[i] = gelu_tanh_f32(gu[m * 2 * n + k]) * gu[m * 2 * n + n + k];
    }
}

__global__ __launch_bounds__(256) void scale_kernel(float* y, float f, int64_t n) {
    for (int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x; i < n; i += (int64_t)gridDim.x * 256) y[i] *= f;
}

// x += alpha * t over rows of the same pitch
__global__ __launch_bounds__(256) void residual_kernel(float* x, const float* t, float alpha, int64_t n) {
    for (int64_t i = (int64_t)blockIdx.x * 256 + threadIdx.x; i < n; i += (int64_t)gridDim.x * 256) x[i] += alpha * t[i];
}

// grid (seqs, parts)
__global__ __launch_bounds__(256) void zero_slots_kernel(const int32_t* slots, float* state, int64_t per_slot) {
    float* s = state + (int64_t)slots[blockIdx.x] * per_slot;
    for (int64_t i = (int64_t)blockIdx.y * 256 + threadIdx.x; i < per_slot; i += (int64_t)gridDim.y * 256) s[i] = 0.f;
}

__global__ __launch_bounds__(1024) void argmax_advance_rows_kernel(const float* logits, int64_t ld, int vocab, int32_t* next, int32_t* tokens,
                                                                   int32_t* pos, int32_t* out, int64_t ld_out) {
    const int b = blockIdx.x;
    const int best = block_argmax_first(logits + (int64_t)b * ld, vocab);
    if (threadIdx.x == 0) {
        const int p = pos[b];
        if (next != nullptr) next[b] = best;
        tokens[b] = best;
        if (out != nullptr) out[(int64_t)b * ld_out + p + 1] = best;
        pos[b] = p + 1;
    }
}

int ew_blocks(int64_t n) {
    const int64_t b = (n + 255) / 256;
    return (int)(b > 4096 ? 4096 : b);
}

enum { kStore = 0, kRelu2 = 1, kResidual = 2, kGeglu = 3, kLogits = 4 };

// y[M, N] (+)= alpha * W norm(x), or what a feed-forward makes of it; alpha: residual_mult (kResidual), logit_scale (kLogits), 1.  x f32 with `norm`, or dtype without
int linear(const mi355_hybrid_model* m, const mi355_proj& w, const void* x, int64_t ldx, const void* norm, int what, void* y, int64_t ldy,
           int y_dtype, int M, hipStream_t s) {
    if (m->dtype == MI355_F32) {
        const float* in = (const float*)x;
        int64_t ld_in = ldx;
        if (norm != nullptr) {
            if (int rc = mi355_rmsnorm(x, ldx, norm, m->norm_dtype, m->eps, m->xn, m->ldx, M, w.K, MI355_F32, MI355_F32, s)) return rc;
            in = m->xn;
            ld_in = m->ldx;
        }
        // (kGeglu: the products lie behind the M hidden rows)
        void* dst = what == kResidual ? (void*)m->tmp : what == kGeglu ? (void*)((float*)y + (int64_t)M * ldy) : y;
        const int64_t ld_dst = what == kResidual ? m->ldx : what == kGeglu ? 2 * ldy : ldy;
        if (int rc = mi355_linear_dense(in, ld_in, w.w, nullptr, dst, ld_dst, M, what == kGeglu ? 2 * w.N : w.N, w.K, MI355_F32, s)) return rc;
        if (what == kGeglu) {  // (ldy = w.N)
            hipLaunchKernelGGL(geglu_kernel, dim3(ew_blocks((int64_t)M * ldy)), dim3(256), 0, s, (const float*)dst, (float*)y, w.N, (int64_t)M * ldy);
            MI355_LAUNCH_CHECK();
        } else if (what == kLogits && m->logit_scale != 1.f) {
            hipLaunchKernelGGL(scale_kernel, dim3(ew_blocks((int64_t)M * ldy)), dim3(256), 0, s, (float*)y, m->logit_scale, (int64_t)M * ldy);
            MI355_LAUNCH_CHECK();
        } else if (what == kRelu2) {  // (ldy = w.N: rows without gaps)
            hipLaunchKernelGGL(relu2_kernel, dim3(ew_blocks((int64_t)M * ldy)), dim3(256), 0, s, (float*)y, (int64_t)M * ldy);
            MI355_LAUNCH_CHECK();
        } else if (what == kResidual) {  // (N = ldx = ldy)
            hipLaunchKernelGGL(residual_kernel, dim3(ew_blocks((int64_t)M * m->ldx)), dim3(256), 0, s, (float*)y, m->tmp, m->residual_mult,
                               (int64_t)M * m->ldx);
            MI355_LAUNCH_CHECK();
        }
        return 0;
    }
    mi355_linear_args a;
    memset(&a, 0, sizeof(a));
    a.fmt = MI355_W_BF16;
    a.R = what == kGeglu ? 2 : 1;
    a.w = w.w;
    a.N = w.N;
    a.K = w.K;
    a.x_dtype = norm != nullptr ? MI355_F32 : MI355_BF16;
    a.ldx = ldx;
    a.norm_scale = norm;
    a.norm_dtype = m->norm_dtype;
    a.eps = m->eps;
    a.epi = what == kResidual ? MI355_EPI_ACCUM : what == kGeglu ? MI355_EPI_GEGLU : MI355_EPI_STORE;
    a.flags = (what == kRelu2 ? MI355_LF_RELU2 : 0) | (m->norm_add != 0.f ? MI355_LF_NORM_ONE : 0);
    a.alpha = what == kResidual ? m->residual_mult : what == kLogits ? m->logit_scale : 1.f;
    a.y_dtype = y_dtype;
    a.ldy = ldy;
    const int most = mi355_linear_max_rows(MI355_W_BF16, w.K, a.R, 0);
    // The weight-streaming kernel up to 8 rows; from there on, and for operands that leave its LDS room for a few rows only, the tiled
    // product (split over K, the operand read in place) moves the weights faster: 4096 x 16512 at 4 / 8 / 16 rows 57 / 118 / 251 us against
    // 28 / 28 / 30, 16512 x 4096 with the norm at 8 / 16 rows 31 / 41 against 35 / 36
    const bool wide = M > 8 || most < M || (M > 2 && norm == nullptr && w.K > 12288 && w.K % 128 == 0);
    if (wide) {
        a.x = x;
        a.y = y;
        a.M = M;
        if (norm != nullptr && w.K % 128 == 0 && ldx % 4 == 0) {
            hipLaunchKernelGGL(norm_rows_kernel, dim3(M), dim3(512), 0, s, (const float*)x, ldx, norm, m->norm_dtype, m->eps, w.K, m->norm_add, m->xb);
            MI355_LAUNCH_CHECK();
            a.x = m->xb;
            a.x_dtype = MI355_BF16;
            a.ldx = w.K;
            a.norm_scale = nullptr;
        }
        return mi355_linear_gemm(&a, m->gemm_ws, (size_t)m->gemm_ws_bytes, s);
    }
    a.x = x;
    a.y = y;
    a.M = M;
    return mi355_linear_fast(&a, s);
}

// between the mixes of a row: not a power of two, so that a row's mixes lie on different memory channels
int64_t mix_stride(const mi355_hybrid_model* m) { return (int64_t)m->max_rows * m->ld_n + 1152; }

int norm_groups(const mi355_hybrid_model* m, const void* scale, const mi355_hybrid_layer* l, const mi355_seq_batch* b, const int32_t* want, int rows,
                hipStream_t s) {
    mi355_norm_args a;
    memset(&a, 0, sizeof(a));
    a.dtype = m->dtype, a.rows = rows, a.width = m->width, a.groups = m->norm_groups;
    a.x = m->x, a.ldx = m->ldx, a.want = want;
    a.eps = m->eps, a.scale = scale;
    a.h = m->dtype == MI355_F32 ? (void*)m->xn : (void*)m->xb, a.ldh = m->ld_n;
    if (l != nullptr && l->n_mix > 0) {
        a.n_mix = l->n_mix, a.mu = l->mu, a.shift = l->shift;
        a.mix = m->mix, a.mix_stride = mix_stride(m);
    }
    return mi355_norm_groups(&a, b, (mi355_stream_t)s);
}

mi355_product product_of(const mi355_hybrid_model* m, const void* x, int64_t ldx, int M, int epi, void* y, int64_t ldy, int y_dtype) {
    mi355_product p;
    memset(&p, 0, sizeof(p));
    p.dtype = m->dtype;
    p.x = x, p.ldx = ldx, p.M = M;
    p.y = y, p.ldy = ldy, p.y_dtype = y_dtype, p.epi = epi;
    p.alpha = 1.f;
    p.ws = m->gemm_ws, p.ws_bytes = m->gemm_ws_bytes;
    return p;
}

// the input projections of a parallel layer, out of its normalised rows and their mixes
int parallel_in(const mi355_hybrid_model* m, const mi355_hybrid_layer& l, int M, hipStream_t s) {
    const bool f32 = m->dtype == MI355_F32;
    const int64_t ldp = l.in.N;
    if (l.n_mix == 0) return mi355_product_run(product_of(m, f32 ? (void*)m->xn : (void*)m->xb, m->ld_n, M, MI355_EPI_STORE, m->proj, ldp, m->dtype), l.in, s);
    const size_t size = dtype_size(m->dtype);
    const int64_t stride = mix_stride(m);
    int i = 0;
    if (!f32 && l.mix_stacked > 1 && !mi355_product_wide(l.mix_w[0], M, 1)) {  // a few rows: every mix's product in one launch
        mi355_linear_args a[5];
        for (; i < l.n_mix; ++i) {
            const bool part = i < l.mix_stacked;
            const mi355_proj& w = l.mix_w[part ? 0 : i];
            const int N = part ? w.N / l.mix_stacked : w.N, K = (w.K + 127) / 128 * 128;
            memset(&a[i], 0, sizeof(a[i]));
            a[i].fmt = MI355_W_BF16, a[i].R = 1, a[i].N = N, a[i].K = K;
            a[i].w = (const char*)w.w + (part ? (int64_t)i * N * K * 2 : 0);
            a[i].x = (const char*)m->mix + i * stride * 2, a[i].x_dtype = MI355_BF16, a[i].M = M, a[i].ldx = m->ld_n;
            a[i].epi = MI355_EPI_STORE, a[i].alpha = 1.f;
            a[i].y = (char*)m->proj + l.mix_at[i] * 2, a[i].y_dtype = MI355_BF16, a[i].ldy = ldp;
        }
        return mi355_linear_fast_jobs(a, l.n_mix, s);
    }
    if (l.mix_stacked > 1) {  // parts of equal size, one stream
        const mi355_proj& w = l.mix_w[0];
        mi355_proj part = w;
        part.N = w.N / l.mix_stacked;
        if (mi355_product_wide(w, M, 1) && part.N % 256 == 0) {
            mi355_product p = product_of(m, m->mix, m->ld_n, M, MI355_EPI_STORE, (char*)m->proj + l.mix_at[0] * size, ldp, m->dtype);
            p.slice_rows = part.N, p.slice_stride = stride;
            if (int rc = mi355_product_run(p, w, s)) return rc;
            i = l.mix_stacked;
        } else {
            for (; i < l.mix_stacked; ++i) {
                part.w = (const char*)w.w + (int64_t)i * part.N * ((w.K + 127) / 128 * 128) * size;
                const mi355_product p = product_of(m, (const char*)m->mix + i * stride * size, m->ld_n, M, MI355_EPI_STORE,
                                                   (char*)m->proj + l.mix_at[i] * size, ldp, m->dtype);
                if (int rc = mi355_product_run(p, part, s)) return rc;
            }
        }
    }
    for (; i < l.n_mix; ++i) {
        const mi355_product p = product_of(m, (const char*)m->mix + i * stride * size, m->ld_n, M, MI355_EPI_STORE,
                                           (char*)m->proj + l.mix_at[i] * size, ldp, m->dtype);
        if (int rc = mi355_product_run(p, l.mix_w[i], s)) return rc;
    }
    return 0;
}

// the pass between two sublayers: the result `t` behind its gate and norm joins the stream; `next`: the norm of what reads it
mi355_join_args join_of(const mi355_hybrid_model* m, int M, const void* next) {
    mi355_join_args a;
    memset(&a, 0, sizeof(a));
    a.dtype = m->dtype, a.rows = M, a.width = m->width, a.eps = m->eps, a.norm_add = m->norm_add;
    a.t = m->tmp, a.ldt = m->ldx;
    a.x = m->x, a.ldx = m->ldx;
    a.next = next, a.h = m->dtype == MI355_F32 ? (void*)m->xn : (void*)m->xb, a.ldh = m->ld_n;
    return a;
}

// the average behind layer run r, and the norm in front of run r + 1 (none behind the last: the head has its own)
void average_of(const mi355_hybrid_model* m, int r, mi355_join_args& a) {
    const int64_t stride = (int64_t)m->max_rows * m->ldx;
    a.stream = m->stream, a.stream_stride = stride, a.stream_out = m->stream + (r + 1) * stride;
    a.n_stream = r + 1, a.average = m->layers[r].average;
    a.next = r + 1 < m->n_runs ? m->layers[r + 1].norm1 : nullptr;
}

// the sublayers of a sandwich layer behind its mixer: gate columns at `gate` of rows of pitch ldp
int sandwich_out(const mi355_hybrid_model* m, int r, const void* gate, int64_t ldp, int M, hipStream_t s) {
    const mi355_hybrid_layer& l = m->layers[r];
    if (l.out_norm != nullptr) {  // state-space outputs in groups
        mi355_norm_args n;
        memset(&n, 0, sizeof(n));
        n.dtype = m->dtype, n.rows = M, n.width = l.out.K, n.groups = l.out_groups;
        n.x = m->mixed, n.ldx = m->ld_mixed, n.eps = m->eps, n.scale = l.out_norm, n.h = l.cat, n.ldh = l.ld_cat;
        if (int rc = mi355_norm_groups(&n, nullptr, (mi355_stream_t)s)) return rc;
    }
    if (int rc = mi355_product_run(product_of(m, l.cat, l.ld_cat, M, MI355_EPI_STORE, m->tmp, m->ldx, MI355_F32), l.out, s)) return rc;
    mi355_join_args a = join_of(m, M, l.norm2);
    a.gate = (const char*)gate + (int64_t)l.gate_at * dtype_size(m->dtype), a.ld_gate = ldp, a.gate_dtype = m->dtype, a.post = l.post1;
    if (l.mlp == MI355_MLP_NONE) average_of(m, r, a);
    if (int rc = mi355_join_rows(&a, (mi355_stream_t)s)) return rc;
    if (l.mlp == MI355_MLP_NONE) return 0;
    const void* h = a.h;
    if (int rc = mi355_product_run(product_of(m, h, m->ld_n, M, MI355_EPI_STORE, m->side, m->ld_side, MI355_F32), l.side, s)) return rc;
    mi355_experts_args e = l.moe;
    e.dtype = m->dtype, e.rows = M, e.eps = m->eps, e.alpha = 1.f;
    e.h = h, e.ldh = m->ld_n, e.logits = m->side + l.logits_at, e.ld_logits = m->ld_side;
    e.out = m->tmp, e.ld_out = m->ldx;
    e.scratch = m->moe_scratch, e.scratch_bytes = m->moe_scratch_bytes;
    if (int rc = mi355_experts(&e, (mi355_stream_t)s)) return rc;
    a = join_of(m, M, nullptr);
    a.gate = m->side, a.ld_gate = m->ld_side, a.gate_dtype = MI355_F32, a.post = l.post2;
    average_of(m, r, a);
    return mi355_join_rows(&a, (mi355_stream_t)s);
}

// hidden row into `cat`, then x += out [mixer | hidden]
int parallel_out(const mi355_hybrid_model* m, const mi355_hybrid_layer& l, int M, hipStream_t s) {
    const bool f32 = m->dtype == MI355_F32;
    if (l.mlp == MI355_MLP_CLAMPGLU) {
        char* hid = (char*)l.cat + (int64_t)l.hid_at * dtype_size(m->dtype);
        if (f32) {  // gate rows, then up rows
            mi355_proj both = l.up;
            both.N *= 2;
            if (int rc = mi355_product_run(product_of(m, m->xn, m->ld_n, M, MI355_EPI_STORE, m->hid, both.N, MI355_F32), both, s)) return rc;
            const int64_t n = (int64_t)M * l.up.N;
            hipLaunchKernelGGL(clampglu_kernel, dim3(ew_blocks(n)), dim3(256), 0, s, (const float*)m->hid, (float*)hid, l.up.N, l.ld_cat, n, l.limit);
            MI355_LAUNCH_CHECK();
        } else {
            mi355_product p = product_of(m, m->xb, m->ld_n, M, MI355_EPI_CLAMPGLU, hid, l.ld_cat, MI355_BF16);
            p.limit = l.limit;
            if (int rc = mi355_product_run(p, l.up, s)) return rc;
        }
    }
    if (f32) {
        if (int rc = mi355_product_run(product_of(m, l.cat, l.ld_cat, M, MI355_EPI_STORE, m->tmp, m->ldx, MI355_F32), l.out, s)) return rc;
        const int64_t n = (int64_t)M * m->ldx;
        hipLaunchKernelGGL(residual_kernel, dim3(ew_blocks(n)), dim3(256), 0, s, m->x, m->tmp, m->residual_mult, n);
        MI355_LAUNCH_CHECK();
        return 0;
    }
    mi355_product p = product_of(m, l.cat, l.ld_cat, M, MI355_EPI_ACCUM, m->x, m->ldx, MI355_F32);
    p.alpha = m->residual_mult;
    return mi355_product_run(p, l.out, s);
}

}  // namespace

extern "C" int mi355_norm_groups(const mi355_norm_args* a, const mi355_seq_batch* b, mi355_stream_t stream) {
    MI355_CHECK_ARG(a && a->x && a->scale && a->h, MI355_E_ARG, "norm_groups: null argument");
    MI355_CHECK_ARG(a->dtype == MI355_F32 || a->dtype == MI355_BF16, MI355_E_DTYPE, "norm_groups: dtype must be f32 or bf16");
    MI355_CHECK_ARG(a->rows > 0 && a->width > 0 && a->groups > 0 && a->groups <= 4096 && a->width % a->groups == 0 && a->ldx >= a->width && a->ldh >= a->width,
                    MI355_E_SHAPE, "norm_groups: %d groups of a row of %d", a->groups, a->width);
    MI355_CHECK_ARG((uintptr_t)a->x % 16 == 0 && a->ldx % 4 == 0 && (uintptr_t)a->h % 16 == 0 && a->ldh % 8 == 0 && (uintptr_t)a->scale % 16 == 0, MI355_E_SHAPE,
                    "norm_groups: rows and scale start at multiples of 16 bytes");
    NormParams p;
    memset(&p, 0, sizeof(p));
    (mi355_norm_args&)p = *a;
    p.size = a->width / a->groups;
    if (a->n_mix > 0) {
        MI355_CHECK_ARG(b && b->row0 && b->count && b->slot && b->pos && b->rows == a->rows && b->max_count > 0 && a->want == nullptr, MI355_E_ARG,
                        "norm_groups: mixes need the batch of their rows");
        MI355_CHECK_ARG(a->n_mix <= 5 && a->mu && a->shift && a->mix && a->mix_stride % 8 == 0 && (uintptr_t)a->mix % 16 == 0 && (uintptr_t)a->mu % 16 == 0 &&
                            (uintptr_t)a->shift % 16 == 0,
                        MI355_E_ARG, "norm_groups: bad mixes");
        p.b = *b;
    }
    hipStream_t s = (hipStream_t)stream;
    if (a->dtype == MI355_F32) a->n_mix > 0 ? launch_norm<float, true>(p, a->rows, s) : launch_norm<float, false>(p, a->rows, s);
    else a->n_mix > 0 ? launch_norm<bf16_t, true>(p, a->rows, s) : launch_norm<bf16_t, false>(p, a->rows, s);
    MI355_LAUNCH_CHECK();
    return 0;
}

bool mi355_product_wide(const mi355_proj& w, int M, int R) {
    const int K = (w.K + 127) / 128 * 128;
    return M > 8 || mi355_linear_max_rows(MI355_W_BF16, K, R, 0) < M || (M > 2 && K > 12288);
}

int mi355_product_run(const mi355_product& p, const mi355_proj& w, hipStream_t s) {
    if (p.dtype == MI355_F32) {
        MI355_CHECK_ARG(p.epi == MI355_EPI_STORE && p.alpha == 1.f && p.y_dtype == MI355_F32, MI355_E_ARG, "product: f32 operands are stored as they are");
        return mi355_linear_dense(p.x, p.ldx, w.w, w.bias, p.y, p.ldy, p.M, w.N, w.K, MI355_F32, s);
    }
    MI355_CHECK_ARG(w.bias == nullptr || p.epi == MI355_EPI_STORE, MI355_E_ARG, "product: a bias belongs to what is stored");
    mi355_linear_args a;
    memset(&a, 0, sizeof(a));
    a.bias = w.bias;
    a.sz_dtype = MI355_F32;
    a.fmt = MI355_W_BF16;
    a.R = is_pair_epi(p.epi) ? 2 : 1;
    a.w = w.w;
    a.N = w.N;
    a.K = (w.K + 127) / 128 * 128;  // (the stream and the operand are padded with zeros)
    a.x = p.x;
    a.x_dtype = MI355_BF16;
    a.M = p.M;
    a.ldx = p.ldx;
    a.epi = p.epi;
    a.alpha = p.alpha;
    a.limit = p.limit;
    a.y = p.y;
    a.y_dtype = p.y_dtype;
    a.ldy = p.ldy;
    a.slice_rows = p.slice_rows;
    a.slice_stride = p.slice_stride;
    MI355_CHECK_ARG(p.ldx >= a.K && p.ldx % 8 == 0, MI355_E_SHAPE, "product: rows of pitch %lld hold no operand of %d columns", (long long)p.ldx, a.K);
    if (p.slice_rows != 0 || mi355_product_wide(w, p.M, a.R)) return mi355_linear_gemm(&a, p.ws, (size_t)p.ws_bytes, s);
    return mi355_linear_fast(&a, s);
}

extern "C" int mi355_hybrid_forward(const mi355_hybrid_model* m, const mi355_seq_batch* b, const int32_t* tokens, const int32_t* want,
                                    int n_want, float* logits, int run_end, mi355_stream_t stream) {
    MI355_CHECK_ARG(m && b && tokens && m->layers && m->x && m->proj && m->att && m->embed, MI355_E_ARG, "hybrid_forward: null argument");
    MI355_CHECK_ARG((m->dtype == MI355_BF16 && m->xb) || (m->dtype == MI355_F32 && m->xn && m->tmp), MI355_E_DTYPE, "hybrid_forward: bad dtype");
    const int M = b->rows;
    MI355_CHECK_ARG(M > 0 && M <= m->max_rows && n_want >= 0 && (want != nullptr ? n_want <= m->max_rows : n_want == 0 || n_want == M),
                    MI355_E_SHAPE, "hybrid_forward: %d rows (of %d), %d wanted", M, m->max_rows, n_want);
    MI355_CHECK_ARG(b->max_count > 1 || b->rows == b->seqs, MI355_E_SHAPE, "hybrid_forward: a decode step has one row per sequence");
    MI355_CHECK_ARG(m->residual_mult != 0.f && m->logit_scale != 0.f, MI355_E_ARG, "hybrid_forward: residual_mult or logit_scale is 0");
    MI355_CHECK_ARG(m->norm_add == 0.f || (m->norm_add == 1.f && m->dtype == MI355_BF16), MI355_E_ARG, "hybrid_forward: norm_add is 0, or 1 in bf16 models");
    MI355_CHECK_ARG(n_want == 0 || run_end < m->n_runs || (logits && m->final_norm), MI355_E_ARG, "hybrid_forward: nowhere to write logits");
    MI355_CHECK_ARG(m->norm_groups == 0 || (m->norm_groups > 0 && m->width % m->norm_groups == 0 && m->norm_add == 0.f && m->norm_dtype == m->dtype && m->ld_n >= (m->width + 127) / 128 * 128 &&
                                            m->ld_n % 8 == 0), MI355_E_SHAPE, "hybrid_forward: bad norm groups %d of width %d", m->norm_groups, m->width);
    for (int r = 0; r < m->n_runs; ++r) {
        const mi355_hybrid_layer& l = m->layers[r];
        MI355_CHECK_ARG(!l.parallel || (m->norm_groups > 0 && l.cat && l.ld_cat >= l.out.K && (l.mlp == MI355_MLP_NONE || l.mlp == MI355_MLP_CLAMPGLU) &&
                                        l.n_mix <= 5 && (l.n_mix == 0 || (l.mu && l.shift && m->mix))),
                        MI355_E_ARG, "hybrid_forward: bad parallel layer (run %d)", r);
        MI355_CHECK_ARG(!l.sandwich || (!l.parallel && m->norm_groups == 0 && m->embed_norm && m->stream && m->tmp && l.cat && l.ld_cat >= l.out.K && l.post1 && l.average &&
                                        (l.mlp == MI355_MLP_NONE || (l.mlp == MI355_MLP_EXPERTS && l.norm2 && l.post2 && m->side && m->ld_side >= l.side.N)) &&
                                        (l.mixer == MI355_MIX_ATTENTION || (l.mixer == MI355_MIX_SSD && m->mixed && m->ld_mixed >= l.out.K && l.out_norm)) &&
                                        m->residual_mult == 1.f && l.sandwich == m->layers[0].sandwich),
                        MI355_E_ARG, "hybrid_forward: bad sandwich layer (run %d)", r);
        MI355_CHECK_ARG(l.sandwich || l.mixer != MI355_MIX_SSD, MI355_E_ARG, "hybrid_forward: a state-space mixer belongs to a sandwich layer (run %d)", r);
        MI355_CHECK_ARG(l.parallel || l.mlp != MI355_MLP_CLAMPGLU, MI355_E_ARG, "hybrid_forward: a clamped gated feed-forward belongs to a parallel layer (run %d)", r);
    }
    hipStream_t s = (hipStream_t)stream;
    if (m->embed_norm != nullptr && m->n_runs > 0) {
        mi355_join_args a = join_of(m, M, m->layers[0].norm1);
        a.tokens = tokens, a.embed = m->embed, a.vocab = m->vocab, a.post = m->embed_norm, a.stream_out = m->stream;
        if (int rc = mi355_join_rows(&a, stream)) return rc;
    } else {
        hipLaunchKernelGGL(embed_rows_kernel, dim3(M), dim3(256), 0, s, tokens, m->embed, m->dtype, m->x, m->width, m->ldx, m->vocab);
        MI355_LAUNCH_CHECK();
    }
    const int runs = run_end < m->n_runs ? run_end : m->n_runs;
    for (int r = 0; r < runs; ++r) {
        const mi355_hybrid_layer& l = m->layers[r];
        const int64_t ldp = l.in.N;
        void* const y = l.mixer == MI355_MIX_SSD ? m->mixed : l.cat != nullptr ? l.cat : m->att;
        const int64_t ldy = l.mixer == MI355_MIX_SSD ? m->ld_mixed : l.cat != nullptr ? l.ld_cat : m->ld_att;
        void* const proj = l.proj_rows != nullptr ? l.proj_rows : m->proj;
        if (l.sandwich) {
            const mi355_product in = product_of(m, m->dtype == MI355_F32 ? (void*)m->xn : (void*)m->xb, m->ld_n, M, MI355_EPI_STORE, proj, ldp, m->dtype);
            if (int rc = mi355_product_run(in, l.in, s)) return rc;
        } else if (l.parallel) {
            if (int rc = norm_groups(m, l.norm1, &l, b, nullptr, M, s)) return rc;
            if (int rc = parallel_in(m, l, M, s)) return rc;
        } else if (int rc = linear(m, l.in, m->x, m->ldx, l.norm1, kStore, m->proj, ldp, m->dtype, M, s)) return rc;
        if (l.mixer == MI355_MIX_ATTENTION) {
            mi355_window_attn_args a = l.attn;
            a.proj = proj;
            a.ld = ldp;
            a.dtype = m->dtype;
            a.y = y;
            a.ldy = ldy;
            a.partials = m->partials;
            a.partials_bytes = m->partials_bytes;
            if (int rc = mi355_window_attention(&a, b, stream)) return rc;
            // a lender's cache rows: behind the last attention of this step that reads the rows they replace
            const int lender = a.role == MI355_KV_BORROWS ? l.kv_lender : r;
            if (a.role != MI355_KV_OWN && m->layers[lender].kv_last == r) {
                a = m->layers[lender].attn;
                a.proj = m->proj;
                a.ld = ldp;
                a.dtype = m->dtype;
                a.y = m->att;
                if (int rc = mi355_window_cache_write(&a, b, stream)) return rc;
            }
        } else if (l.mixer == MI355_MIX_LATENT) {
            mi355_latent_args a = l.latent;
            a.proj = m->proj;
            a.ld = ldp;
            a.dtype = m->dtype;
            a.y = y;
            a.ldy = ldy;
            a.gemm_ws = m->gemm_ws;
            a.gemm_ws_bytes = m->gemm_ws_bytes;
            if (int rc = mi355_latent_attention(&a, b, stream)) return rc;
        } else {
            mi355_recurrent_args a = l.rec;
            a.proj = proj;
            a.ld = ldp;
            a.dtype = m->dtype;
            a.y = y;
            a.ldy = ldy;
            a.scratch = m->rec_scratch;
            a.scratch_bytes = m->rec_scratch_bytes;
            if (int rc = mi355_recurrent(&a, b, stream)) return rc;
        }
        if (l.sandwich) {
            if (int rc = sandwich_out(m, r, proj, ldp, M, s)) return rc;
            continue;
        }
        if (l.parallel) {
            if (int rc = parallel_out(m, l, M, s)) return rc;
            continue;
        }
        if (int rc = linear(m, l.out, m->att, m->ld_att, nullptr, kResidual, m->x, m->ldx, MI355_F32, M, s)) return rc;
        if (l.mlp == MI355_MLP_EXPERTS) {
            mi355_experts_args e = l.moe;
            e.dtype = m->dtype;
            e.rows = M;
            e.norm = l.norm2;
            e.norm_dtype = m->norm_dtype;
            e.norm_add = m->norm_add;
            e.eps = m->eps;
            e.alpha = m->residual_mult;
            e.x = m->x;
            e.ldx = m->ldx;
            e.scratch = m->moe_scratch;
            e.scratch_bytes = m->moe_scratch_bytes;
            if (int rc = mi355_experts(&e, stream)) return rc;
        } else if (l.mlp != MI355_MLP_NONE) {
            const int what = l.mlp == MI355_MLP_GEGLU ? kGeglu : kRelu2;
            if (int rc = linear(m, l.up, m->x, m->ldx, l.norm2, what, m->hid, l.up.N, m->dtype, M, s)) return rc;
            if (int rc = linear(m, l.down, m->hid, l.up.N, nullptr, kResidual, m->x, m->ldx, MI355_F32, M, s)) return rc;
        }
    }
    if (run_end < m->n_runs || n_want == 0) return 0;
    if (m->norm_groups > 0) {
        if (int rc = norm_groups(m, m->final_norm, nullptr, b, want, n_want, s)) return rc;
        mi355_product p = product_of(m, m->dtype == MI355_F32 ? (void*)m->xn : (void*)m->xb, m->ld_n, n_want, MI355_EPI_STORE, logits, m->ld_logits, MI355_F32);
        MI355_CHECK_ARG(m->dtype == MI355_BF16 || m->logit_scale == 1.f, MI355_E_ARG, "hybrid_forward: no logit_scale behind a norm in groups in f32 models");
        p.alpha = m->logit_scale;
        return mi355_product_run(p, m->head, s);
    }
    const float* xh = m->x;
    if (want != nullptr) {
        hipLaunchKernelGGL(gather_rows_kernel, dim3(n_want), dim3(256), 0, s, m->x, want, m->xw, m->ldx);
        MI355_LAUNCH_CHECK();
        xh = m->xw;
    }
    return linear(m, m->head, xh, m->ldx, m->final_norm, kLogits, logits, m->ld_logits, MI355_F32, n_want, s);
}

extern "C" int mi355_hybrid_reset_slots(const mi355_hybrid_model* m, const int32_t* slots, int n, mi355_stream_t stream) {
    MI355_CHECK_ARG(m && slots && n > 0 && m->layers, MI355_E_ARG, "hybrid_reset_slots: bad argument");
    for (int r = 0; r < m->n_runs; ++r) {
        const mi355_hybrid_layer& l = m->layers[r];
        if (l.mixer == MI355_MIX_ATTENTION || l.mixer == MI355_MIX_LATENT) continue;  // (a cache row is written before it can be seen)
        if (l.n_mix > 0) {
            hipLaunchKernelGGL(zero_slots_kernel, dim3(n, 4), dim3(256), 0, (hipStream_t)stream, slots, l.shift, (int64_t)m->width);
            MI355_LAUNCH_CHECK();
        }
        const int64_t per = (int64_t)l.rec.heads * l.rec.dim * l.rec.vdim;
        hipLaunchKernelGGL(zero_slots_kernel, dim3(n, per > 65536 ? 64 : 4), dim3(256), 0, (hipStream_t)stream, slots, l.rec.state, per);
        MI355_LAUNCH_CHECK();
    }
    return 0;
}

extern "C" int mi355_argmax_advance_rows(const float* logits, int64_t ld, int vocab, int seqs, int32_t* next, int32_t* tokens, int32_t* pos,
                                         int32_t* out, int64_t ld_out, mi355_stream_t stream) {
    MI355_CHECK_ARG(logits && tokens && pos && vocab > 0 && seqs > 0, MI355_E_ARG, "argmax_advance_rows: bad argument");
    hipLaunchKernelGGL(argmax_advance_rows_kernel, dim3(seqs), dim3(1024), 0, (hipStream_t)stream, logits, ld, vocab, next, tokens, pos, out,
                       ld_out);
    MI355_LAUNCH_CHECK();
    return 0;
}
