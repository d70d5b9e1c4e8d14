// Causal attention over a sliding window or a chunk: grouped key / value heads, different key and value sizes, interleaved rotation of
// rot_dims dimensions, queries, keys and values over their root mean square (and by factors per dimension), first rows that stay visible, a factor
// and a distance bias per head, bounded scores, a sink in the softmax sum, sigmoid gates per head or per value, values mixed with those of an
// earlier layer.  A slot's cache is, per key head, `kept` rows for the first positions and a ring for the others.  A layer lends
// its keys and values to later ones, which read its cache (and, in a prompt step, its prepared rows).
//
//   window_rows_kernel    one workgroup per (row, key head, split of the keys): decode steps of any size (q and the row's own k are
//                         normalised and rotated here, the cache row is written here: one launch per layer), f32 models, odd head sizes
//   window_tiles_kernel   128 queries of one head per workgroup on the matrix cores (bf16 prompt steps)
//   prepare_keys_kernel   prompt steps: k rows normalised and rotated, v rows normalised in front of either kernel, in place or (a lender's)
//                         to kv_rows
//   ring_write_kernel     prompt steps: the first and the last rows of every portion enter the cache, behind either kernel (which reads
//                         the rows of earlier portions from it) and, of a lender, behind its last borrower
//
// Scores, softmax and weighted values are f32 (the tiles multiply bf16 operands into f32 accumulators).
#include "common.h"

namespace {

typedef __attribute__((ext_vector_type(16))) float f32x16;
typedef __attribute__((ext_vector_type(2))) __bf16 bf16x2_t;

constexpr int kRowThreads = 256;
constexpr int kKeys = 256;        // keys per pass of the row kernel
constexpr int kMaxSplit = 32;     // (<= 64, a lane each) workgroups over the keys of one (row, key head) in a decode step
constexpr double kInvTwoPi = 0.15915494309189533577;

// row of position p in a slot's cache
__device__ __forceinline__ int cache_row(const mi355_window_attn_args& a, int p) { return p < a.kept ? p : a.kept + (p - a.kept) % a.ring; }
// first position of the window or chunk of the row at position p
__device__ __forceinline__ int first_seen(const mi355_window_attn_args& a, int p) { return a.chunked ? p - p % a.window : p - a.window + 1; }
__device__ __forceinline__ float sigmoid_f32(float z) { return 1.0f / (1.0f + expf(-z)); }
__device__ __forceinline__ float cap_score(float s, float cap) { return cap != 0.f ? cap * tanhf(s / cap) : s; }
// element d of key head g's value of `row`, as it is cached (without its norm): with v_first mixed, in f32
template <typename T>
__device__ __forceinline__ float mixed_value(const mi355_window_attn_args& a, int64_t row, int g, int d, float v);

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

template <typename T>
__device__ __forceinline__ float mixed_value(const mi355_window_attn_args& a, int64_t row, int g, int d, float v) {
    return a.v_first == nullptr ? v : (1.0f - a.v_mix) * v + a.v_mix * to_f32<T>(((const T*)a.v_first)[row * a.ld_v_first + g * a.vdim + d]);
}

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
    int n_split, head_tiles, fresh;  // fresh: a decode step
    int own;                         // a decode step of a layer with keys of its own: the row's k is raw and not in the cache yet
    const void *krows, *vrows;       // prepared keys and values of the step's rows, first key head
    int64_t ld_rows;
};

// ------------------------------------------------------------------------------------ row kernel
// HT query heads of one key head per workgroup, VE consecutive elements per load (8: 16-B loads of bf16; 1: any head size).  FRESH: a decode
// step, whose keys all lie in the cache but a row's own
template <typename T, int HT, int VE, bool FRESH>
__global__ __launch_bounds__(kRowThreads, HT <= 4 ? 4 : 2) void window_rows_kernel(const WinParams p) {
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
    float* kn = q + (HT * dim + 3) / 4 * 4;                     // [dim]: the row's own key, as the ring stores it
    float* vn = kn + (dim + 3) / 4 * 4;           // [vdim, padded to VE]: the row's own value where it is mixed or over its root mean square
    float* sc = vn + (vdim + 7) / 8 * 8;          // [kKeys][HT]
    float* stat = sc + HT * kKeys;                // [4][HT]: maximum, sum, correction, slope of the distance bias
    float* red = stat + 4 * HT;                   // [key lanes][HT][columns]: at most kRowThreads HT VE
    __shared__ int s_seq;

    if constexpr (!FRESH) {
        for (int s = tid; s < p.b.seqs; s += kRowThreads)
            if (row >= p.b.row0[s] && row < p.b.row0[s] + p.b.count[s]) s_seq = s;
        __syncthreads();
    }
    const int seq = FRESH ? row : s_seq;
    const int row0 = p.b.row0[seq], pos0 = p.b.pos[seq];
    const int pos = pos0 + (row - row0);
    const T* proj = (const T*)a.proj;
    const T* prow = proj + (int64_t)row * a.ld;
    const int64_t head_row = ((int64_t)p.b.slot[seq] * a.kv_heads + kvh) * (a.kept + a.ring);
    T* kcache = (T*)a.kring + head_row * dim;
    T* vcache = (T*)a.vring + head_row * vdim;

    const unsigned ldk = (unsigned)p.ld_rows;
    const T* kcur = (const T*)p.krows + (int64_t)row0 * ldk + (int64_t)kvh * dim;
    const T* vcur = (const T*)p.vrows + (int64_t)row0 * ldk + (int64_t)kvh * vdim;

    // The visible keys, in order: number g < n_first is position g, the others follow from position w0 on; the last is the row's own.
    // Numbers from g_cur on are rows of the step (a prompt's), those before lie in the cache, in three runs: first positions, ring, ring
    // behind its wrap
    const int n_first = min(a.keep, pos + 1);
    const int w0 = max(first_seen(a, pos), n_first);
    const int n_keys = n_first + pos - w0 + 1;
    const int w_shift = w0 - n_first;                              // position of number g >= n_first, minus g
    const int w_row = w0 < a.kept ? w0 : a.kept + (w0 - a.kept) % a.ring;
    const int row_shift = w_row - n_first;
    const int g_wrap = w0 < a.kept ? 0x7fffffff : n_first + a.kept + a.ring - w_row;  // (the window is no longer than the ring: one wrap at most)
    const int g_cur = pos0 < n_first ? pos0 : max(n_first, pos0 - w_shift);
    auto row_of = [&](int g) { return (unsigned)(g < n_first ? g : g < g_wrap ? g + row_shift : g + row_shift - a.ring); };
    auto step_row = [&](int g) { return (unsigned)((g < n_first ? g : g + w_shift) - pos0); };
    const int step = (n_keys + p.n_split - 1) / p.n_split;
    const int k_begin = split * step, k_end = min(n_keys, k_begin + step);
    const bool owner = FRESH && p.own && k_begin < n_keys && k_end == n_keys;  // this split holds the row's own key
    const bool made_v = a.unit_v || a.v_first != nullptr;                      // ... whose value is not the projection's

    // 32 lanes per head, a pair of values each: over the root mean square, rotated, scaled; a decode step's own key likewise (number nh)
    T* kw = kcache + row_of(n_keys - 1) * (unsigned)dim;
    const int pairs = (dim + 1) / 2;  // (an odd size: the last pair is one value)
    for (int h = tid >> 5; h < nh + (owner ? 1 : 0); h += kRowThreads / 32) {
        const int lane = tid & 31;
        const bool key = h == nh;
        const T* src = key ? prow + a.off_k + (int64_t)kvh * dim : prow + a.off_q + (int64_t)(h0 + h) * dim;
        auto at = [&](int d) { return d < dim ? to_f32<T>(src[d]) : 0.f; };
        constexpr int kHeld = 2;  // pairs of a lane that are loaded once
        float v[kHeld][2], ss = 0.f;
#pragma unroll
        for (int i = 0; i < kHeld; ++i)
#pragma unroll
            for (int e = 0; e < 2; ++e) v[i][e] = at(2 * (lane + 32 * i) + e);
        float f = key ? 1.f : a.head_scale != nullptr ? a.scale * a.head_scale[h0 + h] : a.scale;
        if (a.unit_qk) {
#pragma unroll
            for (int i = 0; i < kHeld; ++i) ss += v[i][0] * v[i][0] + v[i][1] * v[i][1];
            for (int d = 64 * kHeld + lane; d < dim; d += 32) ss += at(d) * at(d);
            f /= sqrtf(group_sum(ss, 32) / (float)dim + a.unit_eps);
        }
        const float* by = key ? a.k_norm : a.q_norm;
        auto put = [&](int pi, float u, float w) {
            if (by != nullptr) {
                u *= by[2 * pi];
                if (2 * pi + 1 < dim) w *= by[2 * pi + 1];
            }
            if (const int ri = pi - a.rot_at / 2; ri >= 0 && 2 * ri < a.rot_dims) {
                float c, s;
                pair_cos_sin(pos, a.inv_freq[ri], c, s);
                const float r = u * c - w * s;
                w = w * c + u * s;
                u = r;
            }
            u *= f, w *= f;
            if (key) {
                const T ru = from_f32<T>(u), rw = from_f32<T>(w);
                kn[2 * pi] = to_f32<T>(ru);
                if (ht == 0) kw[2 * pi] = ru;
                if (2 * pi + 1 < dim) {
                    kn[2 * pi + 1] = to_f32<T>(rw);
                    if (ht == 0) kw[2 * pi + 1] = rw;
                }
            } else {
                q[h * dim + 2 * pi] = u;
                if (2 * pi + 1 < dim) q[h * dim + 2 * pi + 1] = w;
            }
        };
#pragma unroll
        for (int i = 0; i < kHeld; ++i)
            if (lane + 32 * i < pairs) put(lane + 32 * i, v[i][0], v[i][1]);
        for (int pi = lane + 32 * kHeld; pi < pairs; pi += 32) put(pi, at(2 * pi), at(2 * pi + 1));
    }
    if (owner && ht == 0) {
        T* vw = vcache + row_of(n_keys - 1) * (unsigned)vdim;
        const T* vs = prow + a.off_v + (int64_t)kvh * vdim;
        if (!made_v)
            for (int d = tid; d < vdim; d += kRowThreads) vw[d] = vs[d];
    }
    if (owner && made_v && tid < 64) {
        T* vw = vcache + row_of(n_keys - 1) * (unsigned)vdim;
        const T* vs = prow + a.off_v + (int64_t)kvh * vdim;
        float r = 1.f;
        auto value = [&](int d) { return mixed_value<T>(a, row, kvh, d, to_f32<T>(vs[d])); };
        if (a.unit_v) {
            float ss = 0.f;
            for (int d = tid; d < vdim; d += 64) ss += value(d) * value(d);
            r = 1.0f / sqrtf(group_sum(ss, 64) / (float)vdim + a.unit_eps);
        }
        for (int d = tid; d < (vdim + 7) / 8 * 8; d += 64) {
            const T o = from_f32<T>(d < vdim ? value(d) * r : 0.f);
            vn[d] = to_f32<T>(o);
            if (ht == 0 && d < vdim) vw[d] = o;
        }
    }
    if (tid < HT) {  // the sink is a key without a value: a score of its own in the first split
        const bool sink = a.sink != nullptr && split == 0 && tid < nh;
        stat[tid] = sink ? a.sink[h0 + tid] : -INFINITY;
        stat[HT + tid] = sink ? 1.f : 0.f;
        stat[3 * HT + tid] = a.slope != nullptr && tid < nh ? a.slope[h0 + tid] : 0.f;
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
        // ---- scores: 16 lanes per key, four keys per lane group in flight
        const int l16 = tid & 15;
        for (int k4 = tid >> 4; k4 - (tid >> 4) < nk; k4 += 4 * (kRowThreads / 16)) {
            float dot[4][HT];
            const T* src[4];
#pragma unroll
            for (int u = 0; u < 4; ++u) {
                const int g = kb + min(k4 + u * (kRowThreads / 16), nk - 1);
                src[u] = !FRESH && g >= g_cur ? kcur + step_row(g) * ldk : kcache + row_of(g) * (unsigned)dim;
#pragma unroll
                for (int h = 0; h < HT; ++h) dot[u][h] = 0.f;
            }
            for (int d = l16 * VE; d < dim; d += 16 * VE) {
                float kv[4][VE];
#pragma unroll
                for (int u = 0; u < 4; ++u) load_vec(src[u] + d, kv[u]);
#pragma unroll
                for (int h = 0; h < HT; ++h)
                    if (h < nh) {
#pragma unroll
                        for (int e = 0; e < VE; ++e) {
                            const float qv = q[h * dim + d + e];
#pragma unroll
                            for (int u = 0; u < 4; ++u) dot[u][h] += kv[u][e] * qv;
                        }
                    }
            }
#pragma unroll
            for (int u = 0; u < 4; ++u) {
                const int kk = k4 + u * (kRowThreads / 16);
#pragma unroll
                for (int h = 0; h < HT; ++h) dot[u][h] = group_sum(dot[u][h], 16);
                if (l16 == 0 && kk < nk && !(owner && kb + kk == n_keys - 1)) {
                    const int g = kb + kk;
                    const float dist = (float)(pos - (g < n_first ? g : g + w_shift));
#pragma unroll
                    for (int h = 0; h < HT; ++h)
                        if (h < nh) sc[kk * HT + h] = cap_score(dot[u][h], a.softcap) - stat[3 * HT + h] * dist;
                }
            }
        }
        if (owner && kb + nk == n_keys && (tid >> 4) < nh) {  // the row's own key, prepared above: lane group h takes head h
            const int h = tid >> 4;
            float s = 0.f;
            for (int d = l16; d < dim; d += 16) s += kn[d] * q[h * dim + d];
            s = group_sum(s, 16);
            if (l16 == 0) sc[(n_keys - 1 - kb) * HT + h] = cap_score(s, a.softcap);
        }
        __syncthreads();
        // ---- running maximum and sum: one wave per head
        for (int h = tid >> 6; h < nh; h += kRowThreads / 64) {
            const int lane = tid & 63;
            float m = -INFINITY;
            for (int kk = lane; kk < nk; kk += 64) m = fmaxf(m, sc[kk * HT + h]);
            m = wave_max(m);
            const float m_old = stat[h], m_new = fmaxf(m_old, m);
            float l = 0.f;
            for (int kk = lane; kk < nk; kk += 64) {
                const float e = expf(sc[kk * HT + h] - m_new);
                sc[kk * HT + h] = e;
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
            auto add = [&](int kk, auto src) {
                float v[VE], w[HT];
#pragma unroll
                for (int h = 0; h < HT; ++h) w[h] = sc[kk * HT + h];
                load_vec(src + col * VE, v);
#pragma unroll
                for (int h = 0; h < HT; ++h)
                    if (h < nh) {
#pragma unroll
                        for (int e = 0; e < VE; ++e) acc[h][e] += w[h] * v[e];
                    }
            };
            const int nv = owner && kb + nk == n_keys ? nk - 1 : nk;  // (the own value is not in the cache yet)
            if (nv < nk && kl == 0) {
                if (made_v) add(nk - 1, (const float*)vn);
                else add(nk - 1, prow + a.off_v + (int64_t)kvh * vdim);
            }
#pragma unroll 4
            for (int kk = kl; kk < nv; kk += n_kl) {
                const int g = kb + kk;
                const T* src = !FRESH && g >= g_cur ? vcur + step_row(g) * ldk : vcache + row_of(g) * (unsigned)vdim;
                add(kk, src);
            }
        }
        __syncthreads();
    }
    // ---- sum over the key lanes, gate, store
    auto put = [&](int h, int d, float o) {
        if (p.n_split > 1) {
            a.partials[(((int64_t)row * a.heads + h0 + h) * p.n_split + split) * (vdim + 2) + 2 + d] = o;
        } else {
            o /= stat[HT + h];
            if (a.off_g >= 0) o *= sigmoid_f32(to_f32<T>(prow[a.off_g + (a.gate_values ? (h0 + h) * vdim + d : h0 + h)]));
            ((T*)a.y)[(int64_t)row * a.ldy + (int64_t)(h0 + h) * vdim + d] = from_f32<T>(o);
        }
    };
    if (p.n_split > 1 && tid < nh) {
        float* rec = a.partials + (((int64_t)row * a.heads + h0 + tid) * p.n_split + split) * (vdim + 2);
        rec[0] = stat[tid];
        rec[1] = stat[HT + tid];
    }
    // (every key lane's sums to LDS at once: code that runs once per launch is paid for by instruction fetches, so it is kept short)
    const int cols = n_cols * VE;
    if (kl < n_kl) {
#pragma unroll
        for (int h = 0; h < HT; ++h)
#pragma unroll
            for (int e = 0; e < VE; ++e) red[(kl * HT + h) * cols + col * VE + e] = acc[h][e];
    }
    __syncthreads();
    for (int i = tid; i < nh * cols; i += kRowThreads) {
        const int h = i / cols, d = i - h * cols;
        float o = 0.f;
#pragma unroll 4
        for (int k = 0; k < n_kl; ++k) o += red[k * HT * cols + i];
        if (d < vdim) put(h, d, o);
    }
}

// a split decode step: the splits of one (row, head) joined, gated and stored.  grid (heads, rows)
template <typename T>
__global__ __launch_bounds__(128) void window_join_kernel(const WinParams p) {
    const mi355_window_attn_args& a = p.a;
    const int h = blockIdx.x, row = blockIdx.y;
    const float* rec = a.partials + ((int64_t)row * a.heads + h) * p.n_split * (a.vdim + 2);
    __shared__ float wgt[kMaxSplit];
    const int lane = threadIdx.x & 63;  // (every wave joins the maxima and sums: lane = split)
    const bool in = lane < p.n_split;
    const float ms = in ? rec[lane * (a.vdim + 2)] : -INFINITY, ls = in ? rec[lane * (a.vdim + 2) + 1] : 0.f;
    const float m = wave_max(ms);
    const float e = expf(ms - m);
    if ((int)threadIdx.x < p.n_split) wgt[threadIdx.x] = e;
    const T* gates = (const T*)a.proj + (int64_t)row * a.ld + a.off_g;
    float gate = 1.f / group_sum(e * ls, 64);
    if (a.off_g >= 0 && !a.gate_values) gate *= sigmoid_f32(to_f32<T>(gates[h]));
    float each = 0.f;  // (requested ahead of the records; the loop has one turn unless the values are many)
    if (a.off_g >= 0 && a.gate_values && (int)threadIdx.x < a.vdim) each = to_f32<T>(gates[h * a.vdim + threadIdx.x]);
    __syncthreads();
    for (int d = threadIdx.x; d < a.vdim; d += blockDim.x) {
        float o = 0.f;
#pragma unroll 16
        for (int s = 0; s < p.n_split; ++s) o += wgt[s] * rec[s * (a.vdim + 2) + 2 + d];
        if (a.off_g >= 0 && a.gate_values) o *= sigmoid_f32(d < (int)blockDim.x ? each : to_f32<T>(gates[h * a.vdim + d]));
        ((T*)a.y)[(int64_t)row * a.ldy + (int64_t)h * a.vdim + d] = from_f32<T>(o * gate);
    }
}

// ------------------------------------------------------------------------------------ prompt steps: keys, cache
// grid (ceil(max_count * kv_heads / 4), seqs), 256 threads: a wave per (row, key head)
template <typename T>
__global__ __launch_bounds__(256) void prepare_keys_kernel(const WinParams p) {
    const mi355_window_attn_args& a = p.a;
    const int seq = blockIdx.y, it = blockIdx.x * 4 + (threadIdx.x >> 6), lane = threadIdx.x & 63;
    const int i = it / a.kv_heads, g = it - i * a.kv_heads;
    if (i >= p.b.count[seq]) return;
    const int pos = p.b.pos[seq] + i, half = a.rot_dims / 2, rot0 = a.rot_at / 2;
    const int64_t row = p.b.row0[seq] + i;
    const T* src = (const T*)a.proj + row * a.ld;
    const bool moved = a.role == MI355_KV_LENDS;
    const T *k = src + a.off_k + (int64_t)g * a.dim, *v = src + a.off_v + (int64_t)g * a.vdim;
    T *o = (T*)p.krows + row * p.ld_rows + (int64_t)g * a.dim, *vo = (T*)p.vrows + row * p.ld_rows + (int64_t)g * a.vdim;
    if (a.unit_v || a.v_first != nullptr) {
        auto value = [&](int d) { return mixed_value<T>(a, row, g, d, to_f32<T>(v[d])); };
        float r = 1.f;
        if (a.unit_v) {
            float ss = 0.f;
            for (int d = lane; d < a.vdim; d += 64) ss += value(d) * value(d);
            r = 1.0f / sqrtf(group_sum(ss, 64) / (float)a.vdim + a.unit_eps);
        }
        for (int d = lane; d < a.vdim; d += 64) vo[d] = from_f32<T>(value(d) * r);
    } else if (moved) {
        for (int d = lane; d < a.vdim; d += 64) vo[d] = v[d];
    }
    if (!moved && a.rot_dims == 0 && !a.unit_qk) return;
    const int pairs = (a.dim + 1) / 2;  // (an odd size: the last pair is one value)
    const int p0 = lane < pairs ? lane : pairs - 1;
    const float k0 = to_f32<T>(k[2 * p0]), k1 = 2 * p0 + 1 < a.dim ? to_f32<T>(k[2 * p0 + 1]) : 0.f;
    float rms = 1.f;
    if (a.unit_qk) {
        float ss = lane < pairs ? k0 * k0 + k1 * k1 : 0.f;
        for (int d = 128 + lane; d < a.dim; d += 64) {
            const float u = to_f32<T>(k[d]);
            ss += u * u;
        }
        rms = 1.0f / sqrtf(group_sum(ss, 64) / (float)a.dim + a.unit_eps);
    }
    for (int pi = lane; pi < pairs; pi += 64) {
        const bool two = 2 * pi + 1 < a.dim;
        float u = (pi == lane ? k0 : to_f32<T>(k[2 * pi])) * rms, w = (pi == lane ? k1 : two ? to_f32<T>(k[2 * pi + 1]) : 0.f) * rms;
        if (a.k_norm != nullptr) {
            u *= a.k_norm[2 * pi];
            if (two) w *= a.k_norm[2 * pi + 1];
        }
        if (pi >= rot0 && pi - rot0 < half) {
            float c, s;
            pair_cos_sin(pos, a.inv_freq[pi - rot0], c, s);
            const float r = u * c - w * s;
            w = w * c + u * s;
            u = r;
        }
        o[2 * pi] = from_f32<T>(u);
        if (two) o[2 * pi + 1] = from_f32<T>(w);
    }
}

// grid (min(max_count, ring) + kept, seqs): the last `ring` rows of every portion, and those of positions below `kept`
template <typename T>
__global__ __launch_bounds__(256) void ring_write_kernel(const WinParams p, int n_last, int vec) {
    const mi355_window_attn_args& a = p.a;
    const int seq = blockIdx.y, cnt = p.b.count[seq], pos0 = p.b.pos[seq];
    const bool first = (int)blockIdx.x >= n_last;
    const int i = first ? (int)blockIdx.x - n_last - pos0 : cnt - 1 - (int)blockIdx.x;
    if (i < 0 || i >= cnt || (!first && pos0 + i < a.kept)) return;
    const int64_t row = p.b.row0[seq] + i, to = cache_row(a, pos0 + i), rows = a.kept + a.ring;
    const T *ks = (const T*)p.krows + row * p.ld_rows, *vs = (const T*)p.vrows + row * p.ld_rows;
    const int64_t base = (int64_t)p.b.slot[seq] * a.kv_heads;
    if (vec) {  // 16 bytes at a time
        constexpr int V = 16 / sizeof(T);
        const int nk = a.kv_heads * a.dim / V, nv = a.kv_heads * a.vdim / V;
        for (int j = threadIdx.x; j < nk + nv; j += 256) {
            const bool val = j >= nk;
            const int e = (val ? j - nk : j) * V, n = val ? a.vdim : a.dim, g = e / n;
            T* dst = (T*)(val ? a.vring : a.kring) + ((base + g) * rows + to) * n + (e - g * n);
            *(u32x4*)dst = *(const u32x4*)((val ? vs : ks) + e);
        }
        return;
    }
    for (int j = threadIdx.x; j < a.kv_heads * a.dim; j += 256) {
        const int g = j / a.dim, d = j - g * a.dim;
        ((T*)a.kring)[((base + g) * rows + to) * a.dim + d] = ks[j];
    }
    for (int j = threadIdx.x; j < a.kv_heads * a.vdim; j += 256) {
        const int g = j / a.vdim, d = j - g * a.vdim;
        ((T*)a.vring)[((base + g) * rows + to) * a.vdim + d] = vs[j];
    }
}

// ------------------------------------------------------------------------------------ matrix-core tiles (bf16 prompt steps)
// One workgroup: 128 queries of one head, four waves of 32.  Keys in steps of 64: S^T = K Q^T and O^T += V^T P^T on 32x32x16 MFMAs, so a
// lane holds scores and outputs of ONE query (its column).  A key step's K tile [64][D] (16-B columns XOR-swizzled by the key) and V tile
// (transposed to [D][64 keys], the runs of four keys permuted to the order in which a lane's score registers hold them) are loaded into
// registers while the step before is multiplied; keys of earlier portions come from the ring, the rest from the step's own rows.
constexpr int kBQ = 128, kBK = 64;
constexpr int kVtRow = 2 * kBK + 16;  // bytes per row of the transposed V tile

__device__ __forceinline__ uint32_t pack_bf16x2(float a, float b) {
    const bf16x2_t v = {(__bf16)a, (__bf16)b};
    return __builtin_bit_cast(uint32_t, v);
}
__device__ __forceinline__ float max3f(float a, float b, float c) {
    float r;
    asm("v_max3_f32 %0, %1, %2, %3" : "=v"(r) : "v"(a), "v"(b), "v"(c));
    return r;
}
__device__ __forceinline__ float sigmoid_fast(float z) {  // (in front of a rounding to bf16)
    return __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(z * -1.44269504088896340736f));
}
__device__ __forceinline__ float exp2_fast(float x) { return __builtin_amdgcn_exp2f(x); }

// key and value sizes padded to D and DV (multiples of 32).  Wide keys in front of narrow values (D 192) go global -> LDS without registers
// in between, and the values keep one tile: two workgroups fit a CU
template <int D>
constexpr bool kDmaKeys = D == 192;
template <int D, int DV>
constexpr int tiles_lds() { return 2 * kBK * D * 2 + (kDmaKeys<D> ? 1 : 2) * DV * kVtRow; }

template <int D, int DV>
__global__ __launch_bounds__(256, D <= 192 ? 2 : 1) void window_tiles_kernel(const WinParams p) {
    const mi355_window_attn_args& a = p.a;
    extern __shared__ __attribute__((aligned(16))) char smem[];
    constexpr int kCols = D / 8;                       // 16-B columns of a key row
    constexpr int kKItems = kBK * kCols / 256;         // K chunks per thread
    constexpr int kVCols = DV / 8;
    constexpr int kVItems = (16 * kVCols + 255) / 256;  // V items per thread: (run of 4 keys, column)
    constexpr int kKTile = kBK * D * 2, kVTile = DV * kVtRow;
    constexpr bool kPow2 = (kCols & (kCols - 1)) == 0;
    constexpr int kSwz = !kPow2 ? 7 : kCols < 16 ? kCols - 1 : 15;  // (the swizzled column stays in the row: whole groups of 8)
    const int seq = blockIdx.z;
    const int cnt = p.b.count[seq];
    // an XCD (block index mod 8) takes the query blocks of neighbouring heads: their key head stays in its L2
    const int q_blocks = (p.b.max_count + kBQ - 1) / kBQ;
    const int idx = blockIdx.x >> 3, id = (blockIdx.x & 7) * (gridDim.x >> 3) + idx;  // (the grid is a multiple of 8)
    if (id >= q_blocks * a.heads) return;
    // Long query blocks first; every second group of 32 (the CUs of an XCD) runs the other way round, so that of two workgroups that
    // share a CU one walks many keys and one few
    const bool up = 32 % q_blocks == 0 && ((idx >> 5) & 1);
    const int h = id / q_blocks, qb = up ? id % q_blocks : q_blocks - 1 - id % q_blocks;
    if (qb * kBQ >= cnt) return;
    const int kvh = h / (a.heads / a.kv_heads);
    const int row0 = p.b.row0[seq], pos0 = p.b.pos[seq];
    const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
    const int hh = lane >> 5, c = lane & 31;
    const int qi = qb * kBQ + wave * 32 + c;
    const bool q_ok = qi < cnt;
    const int q_row = q_ok ? qi : cnt - 1;
    const int q_pos = pos0 + q_row;
    const bf16_t* proj = (const bf16_t*)a.proj;
    const int q_first = pos0 + qb * kBQ, q_last = pos0 + min(qb * kBQ + kBQ, cnt) - 1;
    // key steps: those of the first `keep` positions that lie in front of the window, then the window's
    const int kb0 = max(0, first_seen(a, q_first)) / kBK, kb1 = q_last / kBK + 1;
    const int n_first = min((a.keep + kBK - 1) / kBK, kb0);
    // the wave's own range, for the masks
    const int w_first = min(pos0 + qb * kBQ + wave * 32, pos0 + cnt - 1), w_last = min(w_first + 31, pos0 + cnt - 1);
    const int q_lo = first_seen(a, q_pos), w_first_lo = first_seen(a, w_first), w_last_lo = first_seen(a, w_last);

    // ---- Q^T operands: q[16 ks + 8 hh .. + 8), rotated, scaled to the exp2 domain, rounded once
    bf16x8 bq[D / 16];
    {
        const bf16_t* src = proj + (int64_t)(row0 + q_row) * a.ld + a.off_q + (int64_t)h * a.dim;
        // (bounded scores: to twice the argument of the tanh in that domain)
        float qs = (a.head_scale != nullptr ? a.scale * a.head_scale[h] : a.scale) * 1.44269504088896340736f * (a.softcap != 0.f ? 2.0f / a.softcap : 1.0f);
        if (a.unit_qk) {  // lanes c and c + 32 hold the row between them
            float ss = 0.f;
#pragma unroll
            for (int ks = 0; ks < D / 16; ++ks) {
                const int d0 = 16 * ks + 8 * hh;
                if (d0 < a.dim) {
                    float v[8];
                    load_vec(src + d0, v);
#pragma unroll
                    for (int e = 0; e < 8; ++e) ss += v[e] * v[e];
                }
            }
            ss += lane_xor32(ss);
            qs /= sqrtf(ss / (float)a.dim + a.unit_eps);
        }
#pragma unroll
        for (int ks = 0; ks < D / 16; ++ks) {
            const int d0 = 16 * ks + 8 * hh;
            u32x4 o = {0u, 0u, 0u, 0u};
            if (d0 < a.dim) {  // (dim % 8 == 0)
                float v[8];
                load_vec(src + d0, v);
#pragma unroll
                for (int e = 0; e < 8; e += 2) {
                    float u = v[e], w = v[e + 1];
                    if (a.q_norm != nullptr) u *= a.q_norm[d0 + e], w *= a.q_norm[d0 + e + 1];
                    if (const int rd = d0 + e - a.rot_at; rd >= 0 && rd < a.rot_dims) {
                        float cs, sn;
                        pair_cos_sin(q_pos, a.inv_freq[rd >> 1], cs, sn);
                        const float r = u * cs - w * sn;
                        w = w * cs + u * sn;
                        u = r;
                    }
                    o[e >> 1] = pack_bf16x2(u * qs, w * qs);
                }
            }
            bq[ks] = __builtin_bit_cast(bf16x8, o);
        }
    }
    const int64_t slot_head = (int64_t)p.b.slot[seq] * a.kv_heads + kvh;
    const bf16_t* kcache = (const bf16_t*)a.kring + slot_head * (a.kept + a.ring) * a.dim;
    const bf16_t* vcache = (const bf16_t*)a.vring + slot_head * (a.kept + a.ring) * a.vdim;
    // rows of the step, from position k_pos0 on; role MI355_KV_ROWS: every position's, the last kdim .. dim of a key from the common tail
    const bool all = a.role == MI355_KV_ROWS;
    const int64_t k_row0 = all ? seq * a.rows_per_seq : row0;
    const int k_pos0 = all ? 0 : pos0, kdim = a.dim - a.tail_dims;
    const bf16_t* kcur = (const bf16_t*)p.krows + k_row0 * p.ld_rows + (int64_t)kvh * kdim;
    const bf16_t* vcur = (const bf16_t*)p.vrows + k_row0 * p.ld_rows + (int64_t)kvh * a.vdim;
    const bf16_t* tail = (const bf16_t*)a.key_tail + (int64_t)p.b.slot[seq] * a.tail_slot - kdim;  // (read from column kdim on)
    const int p_last = pos0 + cnt - 1;
    u32x4 kreg[kDmaKeys<D> ? 1 : kKItems], vreg[kVItems][4];
    const u32x4 zero4 = {0u, 0u, 0u, 0u};
    const int t_key = threadIdx.x / kCols, t_col = threadIdx.x % kCols, t_run = threadIdx.x & 15, t_vcol = threadIdx.x >> 4;
    const bool k_in = t_col * 8 < a.dim;
    constexpr bool kDma = kDmaKeys<D>;
    constexpr int kVTiles = kDma ? 1 : 2;
    // kDma: a thread's chunks of a step, one after the other in LDS (chunk = (key, slot); slot s of a key holds column s ^ (key & kSwz))
    int dkey[kDma ? kKItems : 1], dcol[kDma ? kKItems : 1];
    if constexpr (kDma) {
#pragma unroll
        for (int i = 0; i < kKItems; ++i) {
            const int it = i * 256 + threadIdx.x;
            dkey[i] = it / kCols;
            dcol[i] = ((it % kCols) ^ (dkey[i] & kSwz)) * 8;
            if (dcol[i] >= a.dim) dcol[i] = 0;  // (the query has zeros there: any finite key will do)
        }
    }
    auto dma_keys = [&](int kb, int buf) {
#pragma unroll
        for (int i = 0; i < kKItems; ++i) {
            const int kp = min(kb * kBK + dkey[kDma ? i : 0], p_last), col = dcol[kDma ? i : 0];
            const bf16_t* src = (col >= kdim ? tail + (unsigned)kp * (unsigned)a.ld_tail
                                 : kp >= k_pos0 ? kcur + (unsigned)(kp - k_pos0) * (unsigned)p.ld_rows
                                                : kcache + (unsigned)cache_row(a, kp) * (unsigned)a.dim) + col;
            __builtin_amdgcn_global_load_lds((const __attribute__((address_space(1))) void*)src,
                                             (__attribute__((address_space(3))) void*)(smem + buf * kKTile + (i * 256 + wave * 64) * 16), 16, 0, 0);
        }
    };
    auto load_tile = [&](int kb) {
        if ((kDma || a.tail_dims == 0) && kb * kBK >= k_pos0 && kb * kBK + kBK - 1 <= p_last) {  // all of the step's own rows: one multiply per thread
            const unsigned ld = (unsigned)p.ld_rows;
            const unsigned ko = (unsigned)(kb * kBK + t_key - k_pos0) * ld + t_col * 8;
            if constexpr (!kDma) {
#pragma unroll
                for (int i = 0; i < kKItems; ++i) kreg[i] = *(const u32x4*)(kcur + (k_in ? ko + (unsigned)i * (256 / kCols) * ld : 0u));
            }
            const unsigned vo = (unsigned)(kb * kBK + t_run * 4 - k_pos0) * ld;
#pragma unroll
            for (int i = 0; i < kVItems; ++i) {
                const int col = t_vcol + 16 * i;
                const unsigned o = col * 8 < a.vdim ? vo + col * 8 : 0u;
#pragma unroll
                for (int r = 0; r < 4; ++r) vreg[i][r] = *(const u32x4*)(vcur + (o + (unsigned)r * ld));
            }
            if (!kDma && !k_in) {
#pragma unroll
                for (int i = 0; i < kKItems; ++i) kreg[i] = zero4;
            }
            if (DV != a.vdim) {
#pragma unroll
                for (int i = 0; i < kVItems; ++i)
                    if ((t_vcol + 16 * i) * 8 >= a.vdim) {
#pragma unroll
                        for (int r = 0; r < 4; ++r) vreg[i][r] = zero4;
                    }
            }
            return;
        }
#pragma unroll
        for (int i = 0; i < (kDma ? 0 : kKItems); ++i) {
            const int it = i * 256 + threadIdx.x, key = it / kCols, col = it % kCols;
            const int kp = kb * kBK + key;
            kreg[i] = zero4;
            if (col * 8 < a.dim && kp <= p_last) {
                const bf16_t* src = col * 8 >= kdim ? tail + (int64_t)kp * a.ld_tail
                                    : kp >= k_pos0 ? kcur + (int64_t)(kp - k_pos0) * p.ld_rows
                                                   : kcache + (int64_t)cache_row(a, kp) * a.dim;
                kreg[i] = *(const u32x4*)(src + col * 8);
            }
        }
#pragma unroll
        for (int i = 0; i < kVItems; ++i) {
            const int it = i * 256 + threadIdx.x, run = it & 15, col = it >> 4;
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                const int kp = kb * kBK + run * 4 + r;
                vreg[i][r] = zero4;
                if (col < kVCols && col * 8 < a.vdim && kp <= p_last) {
                    const bf16_t* src = kp >= k_pos0 ? vcur + (int64_t)(kp - k_pos0) * p.ld_rows : vcache + (int64_t)cache_row(a, kp) * a.vdim;
                    vreg[i][r] = *(const u32x4*)(src + col * 8);
                }
            }
        }
    };
    auto store_tile = [&](int buf) {
        char* kt = smem + buf * kKTile;
        char* vt = smem + 2 * kKTile + (buf & (kVTiles - 1)) * kVTile;
#pragma unroll
        for (int i = 0; i < (kDma ? 0 : kKItems); ++i) {
            const int it = i * 256 + threadIdx.x, key = it / kCols, col = it % kCols;
            *(u32x4*)(kt + key * (D * 2) + ((col ^ (key & kSwz)) << 4)) = kreg[i];
        }
#pragma unroll
        for (int i = 0; i < kVItems; ++i) {
            const int it = i * 256 + threadIdx.x, run = it & 15, col = it >> 4;
            if (col >= kVCols) continue;
            const int G = run >> 2, r = run & 3;
            const int pbyte = (G * 16 + 4 * ((r & 1) * 2 + (r >> 1))) * 2;
#pragma unroll
            for (int e = 0; e < 8; ++e) {
                const int dw = e >> 1;
                u32x2 o;
                if (e & 1) {
                    o[0] = __builtin_amdgcn_perm(vreg[i][1][dw], vreg[i][0][dw], 0x07060302u);
                    o[1] = __builtin_amdgcn_perm(vreg[i][3][dw], vreg[i][2][dw], 0x07060302u);
                } else {
                    o[0] = __builtin_amdgcn_perm(vreg[i][1][dw], vreg[i][0][dw], 0x05040100u);
                    o[1] = __builtin_amdgcn_perm(vreg[i][3][dw], vreg[i][2][dw], 0x05040100u);
                }
                *(u32x2*)(vt + (col * 8 + e) * kVtRow + pbyte) = o;
            }
        }
    };
    f32x16 acc[DV / 32];
#pragma unroll
    for (int dt = 0; dt < DV / 32; ++dt)
#pragma unroll
        for (int i = 0; i < 16; ++i) acc[dt][i] = 0.f;
    const float cap2 = a.softcap * 1.44269504088896340736f;
    const float slope2 = a.slope != nullptr ? a.slope[h] * 1.44269504088896340736f : 0.f;
    float m_run = -1.0e30f, l_run = 0.f;
    if (a.sink != nullptr) {  // a key without a value; one of the two lanes of a query counts it
        m_run = a.sink[h] * 1.44269504088896340736f;
        l_run = hh == 0 ? 1.f : 0.f;
    }
    int kb = n_first > 0 ? 0 : kb0, buf = 0;

    if constexpr (kDma) dma_keys(kb, 0);
    load_tile(kb);
    store_tile(0);
    __syncthreads();  // (also waits for the keys on their way to LDS)
    for (; kb < kb1; buf ^= 1) {
        const int next = kb + 1 == n_first ? kb0 : kb + 1;
        if (next < kb1) {
            if constexpr (kDma) dma_keys(next, buf ^ 1);
            load_tile(next);
        }
        const char* kt = smem + buf * kKTile;
        const char* vt = smem + 2 * kKTile + (buf & (kVTiles - 1)) * kVTile;
        // a wave none of whose queries sees this step leaves it out (it still stages the next tile)
        const bool seen = kb * kBK <= w_last && (kb * kBK + kBK - 1 >= w_first_lo || kb * kBK < a.keep);
        if (seen) {
            f32x16 st[2];
#pragma unroll
            for (int t2 = 0; t2 < 2; ++t2)
#pragma unroll
                for (int i = 0; i < 16; ++i) st[t2][i] = 0.f;
#pragma unroll
            for (int ks = 0; ks < D / 16; ++ks)
#pragma unroll
                for (int t2 = 0; t2 < 2; ++t2) {
                    const int key = t2 * 32 + c;
                    const bf16x8 ka = *(const bf16x8*)(kt + key * (D * 2) + (((2 * ks + hh) ^ (key & kSwz)) << 4));
                    st[t2] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(ka, bq[ks], st[t2], 0, 0, 0);
                }
            if (cap2 != 0.f) {  // cap tanh(s / cap), tanh(x) = 1 - 2 / (1 + e^2x)
#pragma unroll
                for (int t2 = 0; t2 < 2; ++t2)
#pragma unroll
                    for (int i = 0; i < 16; ++i) st[t2][i] = cap2 - 2.0f * cap2 * __builtin_amdgcn_rcpf(1.0f + exp2_fast(st[t2][i]));
            }
            if (slope2 != 0.f) {  // (log2 e slope (i - j) is taken off)
                const float at = slope2 * (float)(kb * kBK + 4 * hh - q_pos);
#pragma unroll
                for (int t2 = 0; t2 < 2; ++t2)
#pragma unroll
                    for (int i = 0; i < 16; ++i) st[t2][i] += at + slope2 * (float)(t2 * 32 + (i & 3) + 8 * (i >> 2));
            }
            if (kb * kBK + kBK - 1 > w_first || kb * kBK < w_last_lo) {  // wave-uniform: the step touches an edge
#pragma unroll
                for (int t2 = 0; t2 < 2; ++t2)
#pragma unroll
                    for (int i = 0; i < 16; ++i) {
                        const int kp = kb * kBK + t2 * 32 + (i & 3) + 8 * (i >> 2) + 4 * hh;
                        st[t2][i] = (kp <= q_pos && (kp >= q_lo || kp < a.keep)) ? st[t2][i] : -1.0e30f;
                    }
            }
            // (inline assembly gets no wait states behind the matrix instruction that wrote its operands: 20 here cover the longest)
            asm volatile("s_nop 15\n\ts_nop 3" : "+v"(st[0]), "+v"(st[1]));
            float m_blk = max3f(st[0][0], st[1][0], st[0][1]);  // (v_max3_f32: fmaxf() canonicalises every MFMA result first)
#pragma unroll
            for (int i = 1; i < 16; ++i) m_blk = max3f(m_blk, st[1][i], i < 15 ? st[0][i + 1] : st[1][i]);
            m_blk = max3f(m_blk, lane_xor32(m_blk), m_blk);
            // the reference maximum moves only when it is exceeded by 2^8 (exp2 domain): few steps rescale the outputs.  (A query whose
            // first keys are all masked sums ones at m = -1e30; its first visible key moves m and wipes them out with exp2(-1e30) = 0.)
            const bool move = m_blk > m_run + 8.0f;
            if (__any(move)) {
                const float m_new = move ? m_blk : m_run;
                const float corr = exp2_fast(m_run - m_new);
                l_run *= corr;
                m_run = m_new;
#pragma unroll
                for (int dt = 0; dt < DV / 32; ++dt)
#pragma unroll
                    for (int i = 0; i < 16; ++i) acc[dt][i] *= corr;
            }
            u32x4 pb[2][2];
            float psum = 0.f;
#pragma unroll
            for (int t2 = 0; t2 < 2; ++t2)
#pragma unroll
                for (int i = 0; i < 8; ++i) {
                    const float p0 = exp2_fast(st[t2][2 * i] - m_run), p1 = exp2_fast(st[t2][2 * i + 1] - m_run);
                    psum += p0 + p1;
                    pb[t2][i >> 2][i & 3] = pack_bf16x2(p0, p1);
                }
            l_run += psum;
#pragma unroll
            for (int sg = 0; sg < 4; ++sg) {
                const bf16x8 pf = __builtin_bit_cast(bf16x8, pb[sg >> 1][sg & 1]);
#pragma unroll
                for (int dt = 0; dt < DV / 32; ++dt) {
                    const bf16x8 va = *(const bf16x8*)(vt + (dt * 32 + c) * kVtRow + sg * 32 + hh * 16);
                    acc[dt] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(va, pf, acc[dt], 0, 0, 0);
                }
            }
        }
        if constexpr (kDma) __syncthreads();  // (every wave is done with the step's values)
        if (next < kb1) store_tile(buf ^ 1);
        __syncthreads();
        kb = next;
    }
    const float l = l_run + lane_xor32(l_run);
    if (q_ok) {
        float inv = 1.0f / l;
        const bf16_t* gates = proj + (int64_t)(row0 + q_row) * a.ld + a.off_g;
        if (a.off_g >= 0 && !a.gate_values) inv *= sigmoid_f32(bf16_to_f32(gates[h]));
        const bool each = a.off_g >= 0 && a.gate_values;
        bf16_t* y = (bf16_t*)a.y + (int64_t)(row0 + q_row) * a.ldy + (int64_t)h * a.vdim;
#pragma unroll
        for (int dt = 0; dt < DV / 32; ++dt)
#pragma unroll
            for (int g = 0; g < 4; ++g) {
                const int d = dt * 32 + 8 * g + 4 * hh;
                if (d < a.vdim) {  // (vdim % 8 == 0)
                    float r[4];
#pragma unroll
                    for (int e = 0; e < 4; ++e) r[e] = acc[dt][4 * g + e] * inv;
                    if (each) {
                        const u32x2 z = *(const u32x2*)(gates + h * a.vdim + d);
#pragma unroll
                        for (int e = 0; e < 4; ++e)
                            r[e] *= sigmoid_fast((e & 1) ? __uint_as_float(z[e >> 1] & 0xffff0000u) : __uint_as_float(z[e >> 1] << 16));
                    }
                    u32x2 o;
                    o[0] = pack_bf16x2(r[0], r[1]);
                    o[1] = pack_bf16x2(r[2], r[3]);
                    *(u32x2*)(y + d) = o;
                }
            }
    }
}

template <int D, int DV>
int launch_tiles(const WinParams& p, hipStream_t s) {
    constexpr int lds = tiles_lds<D, DV>();
    static hipError_t e = hipFuncSetAttribute((const void*)window_tiles_kernel<D, DV>, hipFuncAttributeMaxDynamicSharedMemorySize, lds);
    MI355_CHECK_ARG(e == hipSuccess, (int)e, "window_attention: hipFuncSetAttribute failed: %s", hipGetErrorString(e));
    const int q_blocks = (p.b.max_count + kBQ - 1) / kBQ;
    hipLaunchKernelGGL((window_tiles_kernel<D, DV>), dim3((q_blocks * p.a.heads + 7) / 8 * 8, 1, p.b.seqs), dim3(256), lds, s, p);
    MI355_LAUNCH_CHECK();
    return 0;
}

// keys and values of the step's rows and of the cache can be read 16 bytes at a time
bool rows_aligned(const WinParams& p) {
    return p.ld_rows % 8 == 0 && (uintptr_t)p.krows % 16 == 0 && (uintptr_t)p.vrows % 16 == 0 && (uintptr_t)p.a.kring % 16 == 0 &&
           (uintptr_t)p.a.vring % 16 == 0;
}

bool tiles_fit(const WinParams& p) {
    const mi355_window_attn_args& a = p.a;
    return a.dtype == MI355_BF16 && a.dim % 8 == 0 && a.vdim % 8 == 0 && a.dim <= 256 && a.vdim <= 256 && a.ld % 8 == 0 && a.ldy % 4 == 0 &&
           a.off_q % 8 == 0 && rows_aligned(p) && (!a.gate_values || a.off_g % 4 == 0) && (uintptr_t)a.proj % 16 == 0 && (uintptr_t)a.y % 8 == 0;
}

int run_tiles(const WinParams& p, hipStream_t s) {
    const int d = p.a.dim > p.a.vdim ? p.a.dim : p.a.vdim;
    if (d <= 32) return launch_tiles<32, 32>(p, s);
    if (d <= 64) return launch_tiles<64, 64>(p, s);
    if (d <= 128) return launch_tiles<128, 128>(p, s);
    if (p.a.dim <= 192 && p.a.vdim <= 128) return launch_tiles<192, 128>(p, s);
    return launch_tiles<256, 256>(p, s);
}

template <typename T, int HT, int VE, bool FRESH>
int launch_rows_step(const WinParams& p, int rows, hipStream_t s) {
    const size_t red = (size_t)kRowThreads * HT * VE;
    const size_t lds = ((size_t)HT * p.a.dim + p.a.dim + p.a.vdim + 16 + (size_t)HT * kKeys + 4 * HT + red) * 4;
    MI355_CHECK_ARG(lds <= 160 * 1024 - 64, MI355_E_SHAPE, "window_attention: head size %d does not fit LDS", p.a.dim);
    if (lds > 64 * 1024) {
        static hipError_t e = hipFuncSetAttribute((const void*)window_rows_kernel<T, HT, VE, FRESH>, hipFuncAttributeMaxDynamicSharedMemorySize,
                                                  160 * 1024 - 64);
        MI355_CHECK_ARG(e == hipSuccess, (int)e, "window_attention: hipFuncSetAttribute failed: %s", hipGetErrorString(e));
    }
    hipLaunchKernelGGL((window_rows_kernel<T, HT, VE, FRESH>), dim3(p.n_split, p.a.kv_heads * p.head_tiles, rows), dim3(kRowThreads), lds, s, p);
    MI355_LAUNCH_CHECK();
    return 0;
}

template <typename T, int HT, int VE>
int launch_rows(const WinParams& p, int rows, hipStream_t s) {
    return p.fresh ? launch_rows_step<T, HT, VE, true>(p, rows, s) : launch_rows_step<T, HT, VE, false>(p, rows, s);
}

template <typename T>
int run_rows(WinParams p, hipStream_t s) {
    const mi355_window_attn_args& a = p.a;
    const int per = a.heads / a.kv_heads;
    const bool vec = a.dim % 8 == 0 && a.vdim % 8 == 0 && rows_aligned(p);
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
int run_cache_write(const WinParams& p, hipStream_t s) {
    const int n_last = p.b.max_count < p.a.ring ? p.b.max_count : p.a.ring;
    hipLaunchKernelGGL(ring_write_kernel<T>, dim3(n_last + p.a.kept, p.b.seqs), dim3(256), 0, s, p, n_last,
                       p.a.dim % 8 == 0 && p.a.vdim % 8 == 0 && rows_aligned(p));
    MI355_LAUNCH_CHECK();
    return 0;
}

template <typename T>
int run(WinParams p, hipStream_t s) {
    const mi355_window_attn_args& a = p.a;
    if (p.fresh) {
        // splits: enough workgroups for the chip, at least 64 keys each, as far as the scratch goes
        const int per = a.heads / a.kv_heads, ht = per >= 5 ? 8 : per >= 2 ? 4 : 1;
        const int groups = p.b.rows * a.kv_heads * ((per + ht - 1) / ht);
        int n = 2048 / groups;
        const int most = (a.keep + (a.window < a.ring ? a.window : a.ring)) / 64;
        n = n < most ? n : most;
        n = n < kMaxSplit ? n : kMaxSplit;
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
    if (a.role == MI355_KV_LENDS || (a.role == MI355_KV_OWN && (a.rot_dims > 0 || a.unit_qk || a.unit_v || a.v_first != nullptr))) {
        hipLaunchKernelGGL(prepare_keys_kernel<T>, dim3((unsigned)(((int64_t)p.b.max_count * a.kv_heads + 3) / 4), p.b.seqs), dim3(256), 0, s, p);
        MI355_LAUNCH_CHECK();
    }
    p.n_split = 1;
    // (a handful of rows per sequence would leave most of a 128-query tile empty)
    const bool tiles = a.path == 2 || a.role == MI355_KV_ROWS || (a.path == 0 && p.b.max_count > 8);
    if (tiles && tiles_fit(p)) {
        if (int rc = run_tiles(p, s)) return rc;
    } else {
        MI355_CHECK_ARG(a.path != 2 && a.role != MI355_KV_ROWS, MI355_E_SHAPE, "window_attention: the tile kernel takes bf16 heads of up to 256, multiples of 8");
        if (int rc = run_rows<T>(p, s)) return rc;
    }
    return a.role == MI355_KV_OWN ? run_cache_write<T>(p, s) : 0;
}

int make_params(const mi355_window_attn_args* a, const mi355_seq_batch* b, WinParams& p) {
    MI355_CHECK_ARG(a && b && a->proj && a->y && (a->role == MI355_KV_ROWS || (a->kring && a->vring)), MI355_E_ARG, "window_attention: null argument");
    MI355_CHECK_ARG(b->row0 && b->count && b->slot && b->pos, MI355_E_ARG, "window_attention: null batch");
    MI355_CHECK_ARG(b->rows > 0 && b->rows <= 65535 && b->seqs > 0 && b->seqs <= b->rows && b->max_count > 0, MI355_E_SHAPE,
                    "window_attention: bad batch (%d rows, %d sequences)", b->rows, b->seqs);
    MI355_CHECK_ARG(a->dtype == MI355_F32 || a->dtype == MI355_BF16, MI355_E_DTYPE, "window_attention: dtype must be f32 or bf16");
    MI355_CHECK_ARG(a->heads > 0 && a->kv_heads > 0 && a->heads % a->kv_heads == 0 && a->dim > 0 && a->vdim > 0, MI355_E_SHAPE,
                    "window_attention: bad heads %d / %d or sizes %d / %d", a->heads, a->kv_heads, a->dim, a->vdim);
    MI355_CHECK_ARG(a->window > 0 && a->ring > 0 && a->rot_dims >= 0 && a->rot_dims % 2 == 0 && a->rot_at >= 0 && a->rot_at % 2 == 0 && a->rot_at + a->rot_dims <= a->dim &&
                        (a->rot_dims == 0 || a->inv_freq),
                    MI355_E_SHAPE, "window_attention: bad window %d, ring %d or rotation %d", a->window, a->ring, a->rot_dims);
    MI355_CHECK_ARG(a->unit_qk || (a->q_norm == nullptr && a->k_norm == nullptr), MI355_E_ARG, "window_attention: factors per dimension follow a norm");
    MI355_CHECK_ARG(a->softcap >= 0.f && (a->v_first == nullptr || (a->ld_v_first >= (int64_t)a->kv_heads * a->vdim && (a->role == MI355_KV_OWN || a->role == MI355_KV_LENDS))),
                    MI355_E_ARG, "window_attention: bad softcap %g or first values", a->softcap);
    MI355_CHECK_ARG(a->keep >= 0 && a->keep <= a->kept, MI355_E_SHAPE, "window_attention: %d first rows visible, %d cached", a->keep, a->kept);
    MI355_CHECK_ARG(a->role == MI355_KV_ROWS ? b->max_count > 1 && a->rows_per_seq > 0 && a->tail_dims >= 0 && a->tail_dims < a->dim && a->tail_dims % 8 == 0 &&
                                                   (uint64_t)a->rows_per_seq * (uint64_t)a->ld_tail < 0xFFFFFFFFull &&
                                                   a->off_v_rows % 8 == 0 && (a->tail_dims == 0 || (a->key_tail && a->ld_tail % 8 == 0 && a->tail_slot % 8 == 0 &&
                                                                                                    (uintptr_t)a->key_tail % 16 == 0))
                                             : a->tail_dims == 0,
                    MI355_E_ARG, "window_attention: bad rows of all positions");
    MI355_CHECK_ARG(a->role >= MI355_KV_OWN && a->role <= MI355_KV_ROWS && (a->role == MI355_KV_OWN || a->kv_rows), MI355_E_ARG,
                    "window_attention: a lender and its borrowers share kv_rows");
    p.a = *a;
    p.b = *b;
    p.fresh = b->max_count == 1;
    p.own = p.fresh && a->role != MI355_KV_BORROWS;
    p.n_split = p.head_tiles = 1;
    const int size = dtype_size(a->dtype);
    if (a->role == MI355_KV_OWN || p.own) {
        p.krows = (const char*)a->proj + (int64_t)a->off_k * size;
        p.vrows = (const char*)a->proj + (int64_t)a->off_v * size;
        p.ld_rows = a->ld;
    } else if (a->role == MI355_KV_ROWS) {
        p.krows = a->kv_rows;
        p.vrows = (const char*)a->kv_rows + (int64_t)a->off_v_rows * size;
        p.ld_rows = a->ld_rows;
    } else {
        p.krows = a->kv_rows;
        p.vrows = (const char*)a->kv_rows + (int64_t)a->kv_heads * a->dim * size;
        p.ld_rows = (int64_t)a->kv_heads * (a->dim + a->vdim);
    }
    MI355_CHECK_ARG((uint64_t)(a->role == MI355_KV_ROWS ? a->rows_per_seq : b->max_count) * (uint64_t)p.ld_rows < 0xFFFFFFFFull && (uint64_t)b->max_count * (uint64_t)a->ld < 0xFFFFFFFFull &&
                        (uint64_t)(a->kept + (int64_t)a->ring) * (a->dim > a->vdim ? a->dim : a->vdim) < 0xFFFFFFFFull,
                    MI355_E_SHAPE, "window_attention: %d rows of pitch %lld or a cache of %d + %d rows exceed 32-bit offsets", b->max_count,
                    (long long)a->ld, a->kept, a->ring);
    return 0;
}

}  // namespace

extern "C" int mi355_window_attention(const mi355_window_attn_args* a, const mi355_seq_batch* b, mi355_stream_t stream) {
    WinParams p;
    if (int rc = make_params(a, b, p)) return rc;
    return a->dtype == MI355_F32 ? run<float>(p, (hipStream_t)stream) : run<bf16_t>(p, (hipStream_t)stream);
}

extern "C" int mi355_window_cache_write(const mi355_window_attn_args* a, const mi355_seq_batch* b, mi355_stream_t stream) {
    WinParams p;
    if (int rc = make_params(a, b, p)) return rc;
    MI355_CHECK_ARG(a->role == MI355_KV_LENDS, MI355_E_ARG, "window_cache_write: the other layers write their cache themselves");
    if (p.fresh) return 0;  // (a decode step wrote its rows with the lender's attention)
    return a->dtype == MI355_F32 ? run_cache_write<float>(p, (hipStream_t)stream) : run_cache_write<bf16_t>(p, (hipStream_t)stream);
}
