// Causal attention over a sliding window: grouped key / value heads, different key and value sizes, interleaved rotation of the first
// rot_dims dimensions, one sigmoid gate per head.  A slot's cache is a ring of rows per key head.
//
//   window_rows_kernel    one workgroup per (row, key head, split of the keys): decode steps of any size (q and the row's own k are
//                         rotated here, the ring row is written here: one launch per layer), f32 models, odd head sizes
//   window_tiles_kernel   128 queries of one head per workgroup on the matrix cores (bf16 prompt steps)
//   rotate_keys_kernel    prompt steps: k rows rotated in place, in front of either kernel
//   ring_write_kernel     prompt steps: the last rows of every portion enter the ring, behind either kernel (which reads the rows of
//                         earlier portions from it)
//
// Scores, softmax and weighted values are f32 (the tiles multiply bf16 operands into f32 accumulators).
#include "common.h"

namespace {

typedef __attribute__((ext_vector_type(16))) float f32x16;
typedef __attribute__((ext_vector_type(2))) __bf16 bf16x2_t;

constexpr int kRowThreads = 256;
constexpr int kKeys = 256;        // keys per pass of the row kernel
constexpr double kInvTwoPi = 0.15915494309189533577;

// turn of (u, v) by pos * inv_freq: the angle is reduced in f64, so far positions keep f32 accuracy
__device__ __forceinline__ void pair_cos_sin(int pos, double inv_freq, float& c, float& s) {
    double turns = (double)pos * (inv_freq * kInvTwoPi);
    turns -= rint(turns);
    sincospif(2.0f * (float)turns, &s, &c);
}

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

template <typename T, int N>
__device__ __forceinline__ void load_vec(const T* p, float (&o)[N]) {
    if constexpr (N == 8 && sizeof(T) == 2) {
        const u32x4 r = *(const u32x4*)p;
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            o[2 * i] = __uint_as_float(r[i] << 16);
            o[2 * i + 1] = __uint_as_float(r[i] & 0xffff0000u);
        }
    } else if constexpr (N == 8) {
        const f32x4 a = ((const f32x4*)p)[0], b = ((const f32x4*)p)[1];
#pragma unroll
        for (int i = 0; i < 4; ++i) o[i] = a[i], o[4 + i] = b[i];
    } else {
#pragma unroll
        for (int i = 0; i < N; ++i) o[i] = to_f32<T>(p[i]);
    }
}

struct WinParams {
    mi355_window_attn_args a;
    mi355_seq_batch b;
    int n_split, head_tiles, fresh;  // fresh: a decode step (the row's own k is unrotated and not in the ring yet)
};

// ------------------------------------------------------------------------------------ row kernel
// HT query heads of one key head per workgroup, VE consecutive elements per load (8: 16-B loads of bf16; 1: any head size)
template <typename T, int HT, int VE>
__global__ __launch_bounds__(kRowThreads) void window_rows_kernel(const WinParams p) {
    const mi355_window_attn_args& a = p.a;
    extern __shared__ __attribute__((aligned(16))) char smem[];
    const int tid = threadIdx.x;
    const int row = blockIdx.z, split = blockIdx.x;
    const int kvh = blockIdx.y / p.head_tiles, ht = blockIdx.y - kvh * p.head_tiles;
    const int per = a.heads / a.kv_heads;
    const int nh = min(HT, per - ht * HT);        // heads of this workgroup
    const int h0 = kvh * per + ht * HT;
    const int dim = a.dim, vdim = a.vdim;
    float* q = (float*)smem;                      // [HT][dim], scaled
    float* kn = q + HT * dim;                     // [dim]: the row's own key, as the ring stores it
    float* sc = kn + dim;                         // [HT][kKeys]
    float* red = sc + HT * kKeys;                 // [kRowThreads][VE]
    float* stat = red + kRowThreads * VE;         // [3][HT]: maximum, sum, correction
    __shared__ int s_seq;

    if (!p.fresh) {
        for (int s = tid; s < p.b.seqs; s += kRowThreads)
            if (row >= p.b.row0[s] && row < p.b.row0[s] + p.b.count[s]) s_seq = s;
        __syncthreads();
    }
    const int seq = p.fresh ? row : s_seq;
    const int row0 = p.b.row0[seq], pos0 = p.b.pos[seq];
    const int pos = pos0 + (row - row0);
    const T* proj = (const T*)a.proj;
    const T* prow = proj + (int64_t)row * a.ld;
    const T* kring = (const T*)a.kring + ((int64_t)p.b.slot[seq] * a.kv_heads + kvh) * a.ring * dim;
    const T* vring = (const T*)a.vring + ((int64_t)p.b.slot[seq] * a.kv_heads + kvh) * a.ring * vdim;

    const int lo = max(0, pos - a.window + 1);
    const int n_keys = pos - lo + 1;
    const int step = (n_keys + p.n_split - 1) / p.n_split;
    const int k_begin = lo + split * step, k_end = min(pos + 1, k_begin + step);
    const bool owner = k_begin <= pos && k_end == pos + 1;  // this split holds the row's own key

    for (int i = tid; i < nh * dim; i += kRowThreads) {
        const int h = i / dim, d = i - h * dim;
        const T* src = prow + a.off_q + (int64_t)(h0 + h) * dim;
        float v = to_f32<T>(src[d]);
        if (d < a.rot_dims) {
            float c, s;
            pair_cos_sin(pos, a.inv_freq[d >> 1], c, s);
            const float w = to_f32<T>(src[d ^ 1]);
            v = (d & 1) ? v * c + w * s : v * c - w * s;
        }
        q[h * dim + d] = v * a.scale;
    }
    if (p.fresh && owner) {
        T* kw = (T*)a.kring + ((int64_t)p.b.slot[seq] * a.kv_heads + kvh) * a.ring * dim + (int64_t)(pos % a.ring) * dim;
        const T* src = prow + a.off_k + (int64_t)kvh * dim;
        for (int d = tid; d < dim; d += kRowThreads) {
            float v = to_f32<T>(src[d]);
            if (d < a.rot_dims) {
                float c, s;
                pair_cos_sin(pos, a.inv_freq[d >> 1], c, s);
                const float w = to_f32<T>(src[d ^ 1]);
                v = (d & 1) ? v * c + w * s : v * c - w * s;
            }
            const T r = from_f32<T>(v);
            kn[d] = to_f32<T>(r);
            if (ht == 0) kw[d] = r;
        }
        if (ht == 0) {
            T* vw = (T*)a.vring + ((int64_t)p.b.slot[seq] * a.kv_heads + kvh) * a.ring * vdim + (int64_t)(pos % a.ring) * vdim;
            const T* vs = prow + a.off_v + (int64_t)kvh * vdim;
            for (int d = tid; d < vdim; d += kRowThreads) vw[d] = vs[d];
        }
    }
    if (tid < HT) {
        stat[tid] = -INFINITY;
        stat[HT + tid] = 0.f;
    }
    __syncthreads();

    const int n_cols = (vdim + VE - 1) / VE;
    const int n_kl = kRowThreads / n_cols;         // key lanes of the weighted sum
    const int col = tid % n_cols, kl = tid / n_cols;
    float acc[HT][VE];
#pragma unroll
    for (int h = 0; h < HT; ++h)
#pragma unroll
        for (int e = 0; e < VE; ++e) acc[h][e] = 0.f;

    for (int kb = k_begin; kb < k_end; kb += kKeys) {
        const int nk = min(kKeys, k_end - kb);
        // ---- scores: 16 lanes per key
        const int l16 = tid & 15;
        for (int kk = tid >> 4; kk < kKeys; kk += kRowThreads / 16) {
            if (kk - (tid >> 4) >= nk) break;  // (uniform per wave up to the DPP groups: whole 16-lane groups leave together)
            const int kp = kb + min(kk, nk - 1);
            float dot[HT];
#pragma unroll
            for (int h = 0; h < HT; ++h) dot[h] = 0.f;
            if (p.fresh && kp == pos) {
                for (int d = l16; d < dim; d += 16) {
                    const float kv = kn[d];
#pragma unroll
                    for (int h = 0; h < HT; ++h)
                        if (h < nh) dot[h] += kv * q[h * dim + d];
                }
            } else {
                const T* src = kp >= pos0 ? proj + (int64_t)(row0 + kp - pos0) * a.ld + a.off_k + (int64_t)kvh * dim
                                          : kring + (int64_t)(kp % a.ring) * dim;
                for (int d = l16 * VE; d < dim; d += 16 * VE) {
                    float kv[VE];
                    load_vec<T, VE>(src + d, kv);
#pragma unroll
                    for (int h = 0; h < HT; ++h)
                        if (h < nh) {
#pragma unroll
                            for (int e = 0; e < VE; ++e) dot[h] += kv[e] * q[h * dim + d + e];
                        }
                }
            }
#pragma unroll
            for (int h = 0; h < HT; ++h) dot[h] = group_sum(dot[h], 16);
            if (l16 == 0 && kk < nk) {
#pragma unroll
                for (int h = 0; h < HT; ++h)
                    if (h < nh) sc[h * kKeys + kk] = dot[h];
            }
        }
        __syncthreads();
        // ---- running maximum and sum: one wave per head
        for (int h = tid >> 6; h < nh; h += kRowThreads / 64) {
            const int lane = tid & 63;
            float m = -INFINITY;
            for (int kk = lane; kk < nk; kk += 64) m = fmaxf(m, sc[h * kKeys + kk]);
            m = wave_max(m);
            const float m_old = stat[h], m_new = fmaxf(m_old, m);
            float l = 0.f;
            for (int kk = lane; kk < nk; kk += 64) {
                const float e = expf(sc[h * kKeys + kk] - m_new);
                sc[h * kKeys + kk] = e;
                l += e;
            }
            l = wave_sum(l);
            if (lane == 0) {
                const float corr = expf(m_old - m_new);
                stat[h] = m_new;
                stat[HT + h] = stat[HT + h] * corr + l;
                stat[2 * HT + h] = corr;
            }
        }
        __syncthreads();
        // ---- weighted values: VE columns per thread, the keys dealt over n_kl threads
        if (kl < n_kl) {
#pragma unroll
            for (int h = 0; h < HT; ++h) {
                const float corr = h < nh ? stat[2 * HT + h] : 0.f;
#pragma unroll
                for (int e = 0; e < VE; ++e) acc[h][e] *= corr;
            }
            for (int kk = kl; kk < nk; kk += n_kl) {
                const int kp = kb + kk;
                const T* src = kp >= pos0 ? proj + (int64_t)(row0 + kp - pos0) * a.ld + a.off_v + (int64_t)kvh * vdim
                                          : vring + (int64_t)(kp % a.ring) * vdim;
                float v[VE];
                load_vec<T, VE>(src + col * VE, v);
#pragma unroll
                for (int h = 0; h < HT; ++h)
                    if (h < nh) {
                        const float w = sc[h * kKeys + kk];
#pragma unroll
                        for (int e = 0; e < VE; ++e) acc[h][e] += w * v[e];
                    }
            }
        }
        __syncthreads();
    }
    // ---- sum over the key lanes, gate, store
    for (int h = 0; h < HT; ++h) {
        if (h >= nh) break;
        if (kl < n_kl) {
#pragma unroll
            for (int hh = 0; hh < HT; ++hh)
                if (hh == h) {
#pragma unroll
                    for (int e = 0; e < VE; ++e) red[(kl * n_cols + col) * VE + e] = acc[hh][e];
                }
        }
        __syncthreads();
        for (int d = tid; d < vdim; d += kRowThreads) {
            float o = 0.f;
            for (int k = 0; k < n_kl; ++k) o += red[k * n_cols * VE + d];
            if (p.n_split > 1) {
                a.partials[(((int64_t)row * a.heads + h0 + h) * p.n_split + split) * (vdim + 2) + 2 + d] = o;
            } else {
                o /= stat[HT + h];
                if (a.off_g >= 0) o *= 1.0f / (1.0f + expf(-to_f32<T>(prow[a.off_g + h0 + h])));
                ((T*)a.y)[(int64_t)row * a.ldy + (int64_t)(h0 + h) * vdim + d] = from_f32<T>(o);
            }
        }
        if (p.n_split > 1 && tid == 0) {
            float* rec = a.partials + (((int64_t)row * a.heads + h0 + h) * p.n_split + split) * (vdim + 2);
            rec[0] = stat[h];
            rec[1] = stat[HT + h];
        }
        __syncthreads();
    }
}

// a split decode step: the splits of one (row, head) joined, gated and stored.  grid (heads, rows)
template <typename T>
__global__ __launch_bounds__(128) void window_join_kernel(const WinParams p) {
    const mi355_window_attn_args& a = p.a;
    const int h = blockIdx.x, row = blockIdx.y;
    const float* rec = a.partials + ((int64_t)row * a.heads + h) * p.n_split * (a.vdim + 2);
    float m = -INFINITY;
    for (int s = 0; s < p.n_split; ++s) m = fmaxf(m, rec[s * (a.vdim + 2)]);
    float l = 0.f;
    for (int s = 0; s < p.n_split; ++s) l += expf(rec[s * (a.vdim + 2)] - m) * rec[s * (a.vdim + 2) + 1];
    float gate = 1.f / l;
    if (a.off_g >= 0) gate /= 1.0f + expf(-to_f32<T>(((const T*)a.proj)[(int64_t)row * a.ld + a.off_g + h]));
    for (int d = threadIdx.x; d < a.vdim; d += blockDim.x) {
        float o = 0.f;
        for (int s = 0; s < p.n_split; ++s) o += expf(rec[s * (a.vdim + 2)] - m) * rec[s * (a.vdim + 2) + 2 + d];
        ((T*)a.y)[(int64_t)row * a.ldy + (int64_t)h * a.vdim + d] = from_f32<T>(o * gate);
    }
}

// ------------------------------------------------------------------------------------ prompt steps: rotation, ring
// grid (ceil(max_count / 4), seqs), 256 threads: a wave per row
template <typename T>
__global__ __launch_bounds__(256) void rotate_keys_kernel(const WinParams p) {
    const mi355_window_attn_args& a = p.a;
    const int seq = blockIdx.y, i = blockIdx.x * 4 + (threadIdx.x >> 6), lane = threadIdx.x & 63;
    if (i >= p.b.count[seq]) return;
    const int pos = p.b.pos[seq] + i, half = a.rot_dims / 2;
    T* k = (T*)a.proj + (int64_t)(p.b.row0[seq] + i) * a.ld + a.off_k;
    for (int pi = lane; pi < half; pi += 64) {
        float c, s;
        pair_cos_sin(pos, a.inv_freq[pi], c, s);
        for (int g = 0; g < a.kv_heads; ++g) {
            T* kp = k + (int64_t)g * a.dim + 2 * pi;
            const float u = to_f32<T>(kp[0]), v = to_f32<T>(kp[1]);
            kp[0] = from_f32<T>(u * c - v * s);
            kp[1] = from_f32<T>(v * c + u * s);
        }
    }
}

// grid (min(max_count, ring), seqs): the last `ring` rows of every portion
template <typename T>
__global__ __launch_bounds__(256) void ring_write_kernel(const WinParams p) {
    const mi355_window_attn_args& a = p.a;
    const int seq = blockIdx.y, cnt = p.b.count[seq];
    const int i = cnt - 1 - (int)blockIdx.x;
    if (i < 0) return;
    const int slot_row = (p.b.pos[seq] + i) % a.ring;
    const T* src = (const T*)a.proj + (int64_t)(p.b.row0[seq] + i) * a.ld;
    const int64_t base = (int64_t)p.b.slot[seq] * a.kv_heads;
    for (int j = threadIdx.x; j < a.kv_heads * a.dim; j += 256) {
        const int g = j / a.dim, d = j - g * a.dim;
        ((T*)a.kring)[((base + g) * a.ring + slot_row) * a.dim + d] = src[a.off_k + j];
    }
    for (int j = threadIdx.x; j < a.kv_heads * a.vdim; j += 256) {
        const int g = j / a.vdim, d = j - g * a.vdim;
        ((T*)a.vring)[((base + g) * a.ring + slot_row) * a.vdim + d] = src[a.off_v + j];
    }
}

template <typename T, int HT, int VE>
int launch_rows(const WinParams& p, int rows, hipStream_t s) {
    const size_t lds = ((size_t)HT * p.a.dim + p.a.dim + (size_t)HT * kKeys + (size_t)kRowThreads * VE + 3 * HT) * 4;
    MI355_CHECK_ARG(lds <= 160 * 1024 - 64, MI355_E_SHAPE, "window_attention: head size %d does not fit LDS", p.a.dim);
    if (lds > 64 * 1024) {
        static hipError_t e = hipFuncSetAttribute((const void*)window_rows_kernel<T, HT, VE>, hipFuncAttributeMaxDynamicSharedMemorySize,
                                                  160 * 1024 - 64);
        MI355_CHECK_ARG(e == hipSuccess, (int)e, "window_attention: hipFuncSetAttribute failed: %s", hipGetErrorString(e));
    }
    hipLaunchKernelGGL((window_rows_kernel<T, HT, VE>), dim3(p.n_split, p.a.kv_heads * p.head_tiles, rows), dim3(kRowThreads), lds, s, p);
    MI355_LAUNCH_CHECK();
    return 0;
}

template <typename T>
int run_rows(WinParams p, hipStream_t s) {
    const mi355_window_attn_args& a = p.a;
    const int per = a.heads / a.kv_heads;
    const bool vec = a.dim % 8 == 0 && a.vdim % 8 == 0 && a.ld % 8 == 0 && a.off_q % 8 == 0 && a.off_k % 8 == 0 && a.off_v % 8 == 0 &&
                     (uintptr_t)a.proj % 16 == 0 && (uintptr_t)a.kring % 16 == 0 && (uintptr_t)a.vring % 16 == 0;
    MI355_CHECK_ARG(vec ? a.vdim <= 8 * kRowThreads : a.vdim <= kRowThreads, MI355_E_SHAPE,
                    "window_attention: value size %d exceeds the row kernel's %d", a.vdim, vec ? 8 * kRowThreads : kRowThreads);
    const int HT = per >= 5 ? 8 : per >= 2 ? 4 : 1;
    p.head_tiles = (per + HT - 1) / HT;
    if (vec) {
        if (HT == 8) return launch_rows<T, 8, 8>(p, p.b.rows, s);
        if (HT == 4) return launch_rows<T, 4, 8>(p, p.b.rows, s);
        return launch_rows<T, 1, 8>(p, p.b.rows, s);
    }
    if (HT == 8) return launch_rows<T, 8, 1>(p, p.b.rows, s);
    if (HT == 4) return launch_rows<T, 4, 1>(p, p.b.rows, s);
    return launch_rows<T, 1, 1>(p, p.b.rows, s);
}

template <typename T>
int run(WinParams p, hipStream_t s) {
    const mi355_window_attn_args& a = p.a;
    if (p.fresh) {
        // splits: enough workgroups for the chip, at least 64 keys each, as far as the scratch goes
        const int per = a.heads / a.kv_heads, ht = per >= 5 ? 8 : per >= 2 ? 4 : 1;
        const int groups = p.b.rows * a.kv_heads * ((per + ht - 1) / ht);
        int n = 512 / groups;
        n = n < a.ring / 64 ? n : a.ring / 64;
        const uint64_t rec = (uint64_t)p.b.rows * a.heads * (a.vdim + 2) * 4;
        if (a.partials == nullptr) n = 1;
        while (n > 1 && rec * n > a.partials_bytes) n /= 2;
        p.n_split = n < 1 ? 1 : n;
        if (int rc = run_rows<T>(p, s)) return rc;
        if (p.n_split > 1) {
            hipLaunchKernelGGL(window_join_kernel<T>, dim3(a.heads, p.b.rows), dim3(128), 0, s, p);
            MI355_LAUNCH_CHECK();
        }
        return 0;
    }
    if (a.rot_dims > 0) {
        hipLaunchKernelGGL(rotate_keys_kernel<T>, dim3((p.b.max_count + 3) / 4, p.b.seqs), dim3(256), 0, s, p);
        MI355_LAUNCH_CHECK();
    }
    p.n_split = 1;
    if (int rc = run_rows<T>(p, s)) return rc;
    hipLaunchKernelGGL(ring_write_kernel<T>, dim3(p.b.max_count < a.ring ? p.b.max_count : a.ring, p.b.seqs), dim3(256), 0, s, p);
    MI355_LAUNCH_CHECK();
    return 0;
}

}  // namespace

extern "C" int mi355_window_attention(const mi355_window_attn_args* a, const mi355_seq_batch* b, mi355_stream_t stream) {
    MI355_CHECK_ARG(a && b && a->proj && a->kring && a->vring && a->y, MI355_E_ARG, "window_attention: null argument");
    MI355_CHECK_ARG(b->row0 && b->count && b->slot && b->pos, MI355_E_ARG, "window_attention: null batch");
    MI355_CHECK_ARG(b->rows > 0 && b->rows <= 65535 && b->seqs > 0 && b->seqs <= b->rows && b->max_count > 0, MI355_E_SHAPE,
                    "window_attention: bad batch (%d rows, %d sequences)", b->rows, b->seqs);
    MI355_CHECK_ARG(a->dtype == MI355_F32 || a->dtype == MI355_BF16, MI355_E_DTYPE, "window_attention: dtype must be f32 or bf16");
    MI355_CHECK_ARG(a->heads > 0 && a->kv_heads > 0 && a->heads % a->kv_heads == 0 && a->dim > 0 && a->vdim > 0, MI355_E_SHAPE,
                    "window_attention: bad heads %d / %d or sizes %d / %d", a->heads, a->kv_heads, a->dim, a->vdim);
    MI355_CHECK_ARG(a->window > 0 && a->ring > 0 && a->rot_dims >= 0 && a->rot_dims % 2 == 0 && a->rot_dims <= a->dim &&
                        (a->rot_dims == 0 || a->inv_freq),
                    MI355_E_SHAPE, "window_attention: bad window %d, ring %d or rotation %d", a->window, a->ring, a->rot_dims);
    WinParams p;
    p.a = *a;
    p.b = *b;
    p.fresh = b->max_count == 1;
    p.n_split = p.head_tiles = 1;
    return a->dtype == MI355_F32 ? run<float>(p, (hipStream_t)stream) : run<bf16_t>(p, (hipStream_t)stream);
}
