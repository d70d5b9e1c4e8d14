// The forward pass of a layered hybrid model (mi355_hybrid_forward): a host-side walk over the layer runs that enqueues this library's
// linears (gemv.hip for a few rows, gemm.hip above, the exact f32 kernel for f32 models), mixers (window_attention.hip, recurrent.hip) and
// experts (experts.hip).  RMSNorm rides in the consuming linear and the residual sum in the producing one; the residual stream is f32.
#include "common.h"

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

}  // namespace

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
    hipStream_t s = (hipStream_t)stream;
    hipLaunchKernelGGL(embed_rows_kernel, dim3(M), dim3(256), 0, s, tokens, m->embed, m->dtype, m->x, m->width, m->ldx, m->vocab);
    MI355_LAUNCH_CHECK();
    const int runs = run_end < m->n_runs ? run_end : m->n_runs;
    for (int r = 0; r < runs; ++r) {
        const mi355_hybrid_layer& l = m->layers[r];
        const int64_t ldp = l.in.N;
        if (int rc = linear(m, l.in, m->x, m->ldx, l.norm1, kStore, m->proj, ldp, m->dtype, M, s)) return rc;
        if (l.mixer == MI355_MIX_ATTENTION) {
            mi355_window_attn_args a = l.attn;
            a.proj = m->proj;
            a.ld = ldp;
            a.dtype = m->dtype;
            a.y = m->att;
            a.ldy = m->ld_att;
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
        } else {
            mi355_recurrent_args a = l.rec;
            a.proj = m->proj;
            a.ld = ldp;
            a.dtype = m->dtype;
            a.y = m->att;
            a.ldy = m->ld_att;
            a.scratch = m->rec_scratch;
            a.scratch_bytes = m->rec_scratch_bytes;
            if (int rc = mi355_recurrent(&a, b, stream)) return rc;
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
        if (l.mixer == MI355_MIX_ATTENTION) continue;  // (a ring row is written before it can be seen)
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
