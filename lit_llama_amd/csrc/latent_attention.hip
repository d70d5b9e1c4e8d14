// Latent attention: causal attention whose keys and values are products with one cached latent row per position, plus a rotated key tail
// that the heads share.  A slot's cache is [c | tail] per position, in position order.
//
//   latent_prep_kernel     norms of the query latent and of c, rotation of the tail; the cache row is written here
//   (queries: a product, mi355_product_run)
//   absorb_*_kernel        q . uk c = (uk^T q) . c: the query in the latents' space, and its rotated part
//   latent_rows_kernel     attention over the latents, one workgroup per (row, head, split of the keys): any size, f32 and bf16
//   latent_mfma_kernel     the same on the matrix cores, 16 or 32 heads per workgroup: every cached row is read once for all of them
//   latent_out_*_kernel    splits joined, values uv (sum of w c) per head
//   gather_latents_kernel  prompt steps of bf16 models: the latents of every position of a sequence, one below the other, in front of the
//                          product that expands them to keys and values (read by window_attention.hip's tiles)
//
// Norms, rotations, scores and softmax are f32.
#include "product.h"

namespace {

constexpr double kInvTwoPi = 0.15915494309189533577;
constexpr int kMaxSplit = 32;
constexpr int kRec = 4;  // floats in front of a softmax record's values: maximum, sum, two unused

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

// turn by pos * inv_freq: the angle is reduced in f64, so far positions keep f32 accuracy
__device__ __forceinline__ void turn(int pos, double inv_freq, float& u, float& w) {
    double turns = (double)pos * (inv_freq * kInvTwoPi);
    turns -= rint(turns);
    float c, s;
    sincospif(2.0f * (float)turns, &s, &c);
    const float r = u * c - w * s;
    w = w * c + u * s;
    u = r;
}

struct LatParams {
    mi355_latent_args a;
    mi355_seq_batch b;
    int fresh;      // a decode step: row s belongs to sequence s
    int row0;       // first row of this launch
    int n_split;
    int ld_c, ld_cq, ld_qh;  // pitch of a cache row, of cq, and of a head of q / qa's source
    int64_t rows_per_seq;
};

// sequence of a row of the step; all threads of the workgroup take part
__device__ __forceinline__ int seq_of(const LatParams& p, int row, int* shared) {
    if (p.fresh) return row;
    for (int s = threadIdx.x; s < p.b.seqs; s += blockDim.x)
        if (row >= p.b.row0[s] && row < p.b.row0[s] + p.b.count[s]) *shared = s;
    __syncthreads();
    return *shared;
}

// grid (rows), 256 threads; V = 8: bf16 rows of whole 16-B vectors
template <typename T, int V>
__global__ __launch_bounds__(256) void latent_prep_kernel(const LatParams p) {
    const mi355_latent_args& a = p.a;
    __shared__ float red[32];
    __shared__ int s_seq;
    const int row = blockIdx.x, tid = threadIdx.x;
    const T* src = (const T*)a.proj + (int64_t)row * a.ld;
    const T *cq = src + a.off_q, *c = src + a.off_c, *tail = c + a.kv_rank;
    T* oq = (T*)a.cq + (int64_t)row * p.ld_cq;
    // vectors of V values, the query latent's in front of c's; a thread's first two stay in registers
    constexpr int kHeld = 2;
    const int nq = a.q_rank / V, nv = nq + a.kv_rank / V;
    float x[kHeld][V], sq = 0.f, sc = 0.f;
    auto get = [&](int v, float (&f)[V]) {
        const T* at = v < nq ? cq + v * V : c + (v - nq) * V;
        if constexpr (V == 8) {
            const u32x4 r = *(const u32x4*)at;
#pragma unroll
            for (int e = 0; e < 4; ++e) f[2 * e] = __uint_as_float(r[e] << 16), f[2 * e + 1] = __uint_as_float(r[e] & 0xffff0000u);
        } else {
            f[0] = to_f32<T>(at[0]);
        }
    };
    auto add = [&](int v, const float (&f)[V]) {
        float t = 0.f;
#pragma unroll
        for (int e = 0; e < V; ++e) t += f[e] * f[e];
        if (v < nq) sq += t;
        else sc += t;
    };
#pragma unroll
    for (int i = 0; i < kHeld; ++i)
        if (tid + 256 * i < nv) get(tid + 256 * i, x[i]);
    float u0 = 0.f, w0 = 0.f;
    if (tid < a.rot_dim / 2) u0 = to_f32<T>(tail[2 * tid]), w0 = to_f32<T>(tail[2 * tid + 1]);
    // (the row is on its way while its sequence is looked up)
    const int seq = seq_of(p, row, &s_seq);
    const int pos = p.b.pos[seq] + row - p.b.row0[seq];
    T* o = (T*)a.cache + ((int64_t)p.b.slot[seq] * a.cache_rows + pos) * p.ld_c;
#pragma unroll
    for (int i = 0; i < kHeld; ++i)
        if (tid + 256 * i < nv) add(tid + 256 * i, x[i]);
    for (int v = tid + 256 * kHeld; v < nv; v += 256) {
        float f[V];
        get(v, f);
        add(v, f);
    }
    sq = group_sum(sq, 64);
    sc = group_sum(sc, 64);
    if ((tid & 63) == 0) red[tid >> 6] = sq, red[4 + (tid >> 6)] = sc;
    __syncthreads();
    const float rq = 1.0f / sqrtf((red[0] + red[1] + red[2] + red[3]) / (float)a.q_rank + a.eps);
    const float rc = 1.0f / sqrtf((red[4] + red[5] + red[6] + red[7]) / (float)a.kv_rank + a.eps);
    auto put = [&](int v, const float (&f)[V]) {
        const bool isq = v < nq;
        const int k = (isq ? v : v - nq) * V;
        const float* w = (isq ? a.q_norm : a.c_norm) + k;
        const float r = isq ? rq : rc;
        T* at = (isq ? oq : o) + k;
        if constexpr (V == 8) {
            u32x4 b;
#pragma unroll
            for (int e = 0; e < 4; ++e)
                b[e] = (uint32_t)f32_to_bf16(f[2 * e] * r * w[2 * e]) | ((uint32_t)f32_to_bf16(f[2 * e + 1] * r * w[2 * e + 1]) << 16);
            *(u32x4*)at = b;
        } else {
            at[0] = from_f32<T>(f[0] * r * w[0]);
        }
    };
#pragma unroll
    for (int i = 0; i < kHeld; ++i)
        if (tid + 256 * i < nv) put(tid + 256 * i, x[i]);
    for (int v = tid + 256 * kHeld; v < nv; v += 256) {
        float f[V];
        get(v, f);
        put(v, f);
    }
    for (int k = a.q_rank + tid; k < p.ld_cq; k += 256) oq[k] = from_f32<T>(0.f);
    o += a.kv_rank;
    for (int i = tid; i < a.rot_dim / 2; i += 256) {
        float u = i == tid ? u0 : to_f32<T>(tail[2 * i]), w = i == tid ? w0 : to_f32<T>(tail[2 * i + 1]);
        turn(pos, a.inv_freq[i], u, w);
        o[2 * i] = from_f32<T>(u);
        o[2 * i + 1] = from_f32<T>(w);
    }
}

// ------------------------------------------------------------------------------------ queries in the latents' space
// grid (heads, rows), 256 threads
template <typename T>
__global__ __launch_bounds__(256) void absorb_rows_kernel(const LatParams p) {
    const mi355_latent_args& a = p.a;
    extern __shared__ __attribute__((aligned(16))) float sm[];
    __shared__ int s_seq;
    const int h = blockIdx.x, row = p.row0 + blockIdx.y, tid = threadIdx.x, seq = seq_of(p, row, &s_seq);
    const int pos = p.b.pos[seq] + row - p.b.row0[seq];
    const T* q = (const T*)a.q + (int64_t)row * a.uq.N + (int64_t)h * p.ld_qh;
    T* o = (T*)a.qa + ((int64_t)row * a.heads + h) * p.ld_c;
    for (int d = tid; d < a.dim; d += 256) sm[d] = to_f32<T>(q[d]);
    __syncthreads();
    for (int r = tid; r < a.kv_rank; r += 256) {
        const T* w = (const T*)a.uk_t + ((int64_t)h * a.kv_rank + r) * a.dim;
        float s = 0.f;
        for (int d = 0; d < a.dim; ++d) s += to_f32<T>(w[d]) * sm[d];
        o[r] = from_f32<T>(s);
    }
    for (int i = tid; i < a.rot_dim / 2; i += 256) {
        float u = to_f32<T>(q[a.dim + 2 * i]), w = to_f32<T>(q[a.dim + 2 * i + 1]);
        turn(pos, a.inv_freq[i], u, w);
        o[a.kv_rank + 2 * i] = from_f32<T>(u);
        o[a.kv_rank + 2 * i + 1] = from_f32<T>(w);
    }
}

// grid (heads, 64-column blocks of the latent + 1, 16-row tiles), 256 threads; dim, kv_rank multiples of 8.  The last block of y rotates
__global__ __launch_bounds__(256) void absorb_mfma_kernel(const LatParams p, int rows) {
    const mi355_latent_args& a = p.a;
    const int h = blockIdx.x, t0 = p.row0 + blockIdx.z * 16, tid = threadIdx.x;
    const int end = p.row0 + rows;
    if (blockIdx.y == gridDim.y - 1) {
        __shared__ int seq16[16];
        if (tid < 16) seq16[tid] = t0 + tid;
        __syncthreads();
        if (!p.fresh) {
            for (int s = tid; s < p.b.seqs; s += 256) {
                const int r0 = p.b.row0[s], r1 = r0 + p.b.count[s];
                for (int t = max(r0, t0); t < min(r1, t0 + 16); ++t) seq16[t - t0] = s;
            }
            __syncthreads();
        }
        const int half = a.rot_dim / 2;
        for (int it = tid; it < 16 * half; it += 256) {
            const int t = it / half, i = it - t * half, row = t0 + t;
            if (row >= end) continue;
            const int seq = seq16[t], pos = p.b.pos[seq] + row - p.b.row0[seq];
            const bf16_t* q = (const bf16_t*)a.q + (int64_t)row * a.uq.N + (int64_t)h * p.ld_qh + a.dim;
            bf16_t* o = (bf16_t*)a.qa + ((int64_t)row * a.heads + h) * p.ld_c + a.kv_rank;
            float u = bf16_to_f32(q[2 * i]), w = bf16_to_f32(q[2 * i + 1]);
            turn(pos, a.inv_freq[i], u, w);
            o[2 * i] = f32_to_bf16(u);
            o[2 * i + 1] = f32_to_bf16(w);
        }
        return;
    }
    const int lane = tid & 63, wave = tid >> 6, c = lane & 15, g = lane >> 4;
    const int r0 = blockIdx.y * 64 + wave * 16;
    if (r0 >= a.kv_rank) return;
    const int row = min(t0 + c, end - 1);
    const bf16_t* w = (const bf16_t*)a.uk_t + ((int64_t)h * a.kv_rank + min(r0 + c, a.kv_rank - 1)) * a.dim;
    const bf16_t* q = (const bf16_t*)a.q + (int64_t)row * a.uq.N + (int64_t)h * p.ld_qh;
    f32x4 acc = {0.f, 0.f, 0.f, 0.f};
    const u32x4 zero = {0u, 0u, 0u, 0u};
    for (int d0 = 8 * g; d0 - 8 * g < a.dim; d0 += 128) {  // four operand pairs in flight
        u32x4 av[4], bv[4];
#pragma unroll
        for (int j = 0; j < 4; ++j) {
            const int d = d0 + 32 * j;
            av[j] = d < a.dim ? *(const u32x4*)(w + d) : zero;
            bv[j] = d < a.dim ? *(const u32x4*)(q + d) : zero;
        }
#pragma unroll
        for (int j = 0; j < 4; ++j)
            acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8, av[j]), __builtin_bit_cast(bf16x8, bv[j]), acc, 0, 0, 0);
    }
    if (t0 + c < end && r0 + 4 * g < a.kv_rank) {
        u32x2 o;
        o[0] = (uint32_t)f32_to_bf16(acc[0]) | ((uint32_t)f32_to_bf16(acc[1]) << 16);
        o[1] = (uint32_t)f32_to_bf16(acc[2]) | ((uint32_t)f32_to_bf16(acc[3]) << 16);
        *(u32x2*)((bf16_t*)a.qa + ((int64_t)(t0 + c) * a.heads + h) * p.ld_c + r0 + 4 * g) = o;
    }
}

// ------------------------------------------------------------------------------------ attention over the latents
// keys [begin, end) of a split: whole steps of 64
__device__ __forceinline__ void split_range(int n_keys, int n_split, int split, int& begin, int& end) {
    const int step = ((n_keys + n_split - 1) / n_split + 63) / 64 * 64;
    begin = split * step;
    end = min(n_keys, begin + step);
}
__device__ __forceinline__ float* record(const LatParams& p, int row, int h, int split) {
    return p.a.partials + (((int64_t)(row - p.row0) * p.a.heads + h) * p.n_split + split) * (p.a.kv_rank + kRec);
}

// grid (splits, heads, rows), 256 threads
template <typename T>
__global__ __launch_bounds__(256) void latent_rows_kernel(const LatParams p) {
    const mi355_latent_args& a = p.a;
    extern __shared__ __attribute__((aligned(16))) float sm[];
    __shared__ int s_seq;
    __shared__ float red[32];
    constexpr int kKeys = 256, kCols = 4;  // (kv_rank <= 1024)
    const int split = blockIdx.x, h = blockIdx.y, row = p.row0 + blockIdx.z, tid = threadIdx.x, seq = seq_of(p, row, &s_seq);
    const int pos = p.b.pos[seq] + row - p.b.row0[seq];
    const int DK = a.kv_rank + a.rot_dim;
    float* q = sm;         // [DK]
    float* sc = sm + DK;   // [kKeys]
    const T* qa = (const T*)a.qa + ((int64_t)row * a.heads + h) * p.ld_c;
    for (int d = tid; d < DK; d += 256) q[d] = to_f32<T>(qa[d]);
    const T* cache = (const T*)a.cache + (int64_t)p.b.slot[seq] * a.cache_rows * p.ld_c;
    int begin, end;
    split_range(pos + 1, p.n_split, split, begin, end);
    float m = split == 0 ? a.sink[h] : -1.0e30f, l = split == 0 ? 1.f : 0.f;  // (the sink is a key without a value)
    float acc[kCols] = {0.f, 0.f, 0.f, 0.f};
    __syncthreads();
    for (int kb = begin; kb < end; kb += kKeys) {
        const int nk = min(kKeys, end - kb), l16 = tid & 15;
        for (int k = tid >> 4; k < nk; k += 16) {
            const T* c = cache + (int64_t)(kb + k) * p.ld_c;
            float s = 0.f;
            for (int d = l16; d < DK; d += 16) s += q[d] * to_f32<T>(c[d]);
            s = group_sum(s, 16);
            if (l16 == 0) sc[k] = s * a.scale;
        }
        __syncthreads();
        const float s = tid < nk ? sc[tid] : -1.0e30f;
        const float m_new = fmaxf(m, block_max(s, red));
        const float e = tid < nk ? expf(s - m_new) : 0.f, corr = expf(m - m_new);
        if (tid < nk) sc[tid] = e;
        l = l * corr + block_sum(e, red);  // (its barriers order the weights in front of the sums below)
        m = m_new;
#pragma unroll
        for (int j = 0; j < kCols; ++j) acc[j] *= corr;
        for (int k = 0; k < nk; ++k) {
            const T* c = cache + (int64_t)(kb + k) * p.ld_c;
            const float w = sc[k];
#pragma unroll
            for (int j = 0; j < kCols; ++j)
                if (tid + 256 * j < a.kv_rank) acc[j] += w * to_f32<T>(c[tid + 256 * j]);
        }
        __syncthreads();
    }
    float* rec = record(p, row, h, split);
    if (tid == 0) rec[0] = m, rec[1] = l;
#pragma unroll
    for (int j = 0; j < kCols; ++j)
        if (tid + 256 * j < a.kv_rank) rec[kRec + tid + 256 * j] = acc[j];
}

// One workgroup: 16 NH heads of one row over a split of its keys, in steps of 64.  S = C Q^T on 16x16x32 MFMAs (a wave per 16 keys and 16
// heads), weights through LDS, O^T += C^T P^T with the latents' columns dealt over the waves in blocks of 32 (RB per wave): the transposed
// operand is read from the same LDS tile as pairs of columns.  The next step's rows are requested while this one is multiplied.
// grid (splits, head tiles, rows), 512 threads
constexpr int kStep = 64;
template <int RB>
constexpr int kTileItems = 4 * RB + 2;  // 16-B chunks per thread and step: kv_rank + rot_dim <= 64 of them
__host__ __device__ constexpr int pad32(int n) { return (n + 31) / 32 * 32; }
__host__ __device__ constexpr int mfma_pitch(int dk) { return pad32(dk) + 8; }
template <int NH>
size_t mfma_lds(int dk) { return (size_t)(kStep + 16 * NH) * mfma_pitch(dk) * 2 + (size_t)16 * NH * (kStep + 8) * 2 + (size_t)16 * NH * 9 * 4; }

template <int NH, int RB>
__global__ __launch_bounds__(512) void latent_mfma_kernel(const LatParams p) {
    const mi355_latent_args& a = p.a;
    extern __shared__ __attribute__((aligned(16))) char smem[];
    __shared__ int s_seq;
    const int split = blockIdx.x, h0 = blockIdx.y * 16 * NH, row = p.row0 + blockIdx.z, tid = threadIdx.x, seq = seq_of(p, row, &s_seq);
    const int pos = p.b.pos[seq] + row - p.b.row0[seq];
    const int R = a.kv_rank, DK = R + a.rot_dim, DKp = pad32(DK), P = mfma_pitch(DK), PP = kStep + 8;
    bf16_t* ks = (bf16_t*)smem;             // [64][P]
    bf16_t* qs = ks + kStep * P;            // [16 NH][P]
    bf16_t* ps = qs + 16 * NH * P;          // [16 NH][PP]
    float* wm = (float*)(ps + 16 * NH * PP);  // [4][16 NH] maxima of the key tiles, sums at the end
    float* cr = wm + 4 * 16 * NH;           // [16 NH] correction of the step
    const int lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), c = lane & 15, g = lane >> 4;
    const int kt = wave & 3, hn = wave >> 2;
    const bool scores = hn < NH;
    int begin, end;
    split_range(pos + 1, p.n_split, split, begin, end);

    const bf16_t* cache = (const bf16_t*)a.cache + (int64_t)p.b.slot[seq] * a.cache_rows * p.ld_c;
    const int cols = DK / 8, items = kStep * cols;
    u32x4 reg[kTileItems<RB>];
    int key_of[kTileItems<RB>], at[kTileItems<RB>];  // a thread's chunks of a step: key, place in the LDS tile
    {
        const int dk = 512 / cols, dc = 512 - dk * cols;
        int key = tid / cols, col = tid - key * cols;
#pragma unroll
        for (int i = 0; i < kTileItems<RB>; ++i) {
            const bool in = tid + 512 * i < items;
            key_of[i] = in ? key : 0x3fffffff;
            at[i] = in ? key * P + col * 8 : 0;
            key += dk, col += dc;
            if (col >= cols) ++key, col -= cols;
        }
    }
    auto load = [&](int kb) {
        const bf16_t* src = cache + (int64_t)kb * p.ld_c;
#pragma unroll
        for (int i = 0; i < kTileItems<RB>; ++i)  // (an LDS row is P elements, a cache row ld_c)
            reg[i] = key_of[i] < end - kb ? *(const u32x4*)(src + (at[i] - key_of[i] * (P - p.ld_c))) : u32x4{0u, 0u, 0u, 0u};
    };
    auto store = [&]() {
#pragma unroll
        for (int i = 0; i < kTileItems<RB>; ++i)
            if (key_of[i] < kStep) *(u32x4*)(ks + at[i]) = reg[i];
    };
    if (begin < end) load(begin);
    for (int it = tid; it < 16 * NH * cols; it += 512) {
        const int h = it / cols, col = it - h * cols;
        *(u32x4*)(qs + h * P + col * 8) =
            h0 + h < a.heads ? *(const u32x4*)((const bf16_t*)a.qa + ((int64_t)row * a.heads + h0 + h) * p.ld_c + col * 8) : u32x4{0u, 0u, 0u, 0u};
    }
    for (int it = tid; it < (kStep + 16 * NH) * (DKp - DK); it += 512) {  // padding columns of keys and queries
        const int r = it / (DKp - DK);
        ks[r * P + DK + it - r * (DKp - DK)] = 0;
    }
    const int head = h0 + hn * 16 + c;
    const bool sink = split == 0 && scores && head < a.heads;
    float m_run = sink ? a.sink[head] : -1.0e30f;
    float l_run = sink && kt == 0 && g == 0 ? 1.f : 0.f;  // (one lane of the head counts the sink)
    f32x4 acc[RB][2][NH];
#pragma unroll
    for (int b = 0; b < RB; ++b)
#pragma unroll
        for (int o = 0; o < 2; ++o)
#pragma unroll
            for (int n = 0; n < NH; ++n) acc[b][o][n] = f32x4{0.f, 0.f, 0.f, 0.f};

    for (int kb = begin; kb < end; kb += kStep) {
        store();
        __syncthreads();
        if (kb + kStep < end) load(kb + kStep);
        f32x4 s = {0.f, 0.f, 0.f, 0.f};
        if (scores) {
            f32x4 s2 = {0.f, 0.f, 0.f, 0.f};
            const bf16_t* ka = ks + (kt * 16 + c) * P + 8 * g;
            const bf16_t* qb = qs + (hn * 16 + c) * P + 8 * g;
            for (int d = 0; d < DKp; d += 64) {
                s = __builtin_amdgcn_mfma_f32_16x16x32_bf16(*(const bf16x8*)(ka + d), *(const bf16x8*)(qb + d), s, 0, 0, 0);
                if (d + 32 < DKp) s2 = __builtin_amdgcn_mfma_f32_16x16x32_bf16(*(const bf16x8*)(ka + d + 32), *(const bf16x8*)(qb + d + 32), s2, 0, 0, 0);
            }
            float m = -1.0e30f;
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                s[r] = kb + kt * 16 + 4 * g + r < end ? (s[r] + s2[r]) * a.scale : -1.0e30f;
                m = fmaxf(m, s[r]);
            }
            m = fmaxf(m, lane_xor16(m));
            m = fmaxf(m, lane_xor32(m));
            if (g == 0) wm[kt * 16 * NH + hn * 16 + c] = m;
        }
        __syncthreads();
        if (scores) {
            float m_new = m_run;
#pragma unroll
            for (int t = 0; t < 4; ++t) m_new = fmaxf(m_new, wm[t * 16 * NH + hn * 16 + c]);
            const float corr = expf(m_run - m_new);
            m_run = m_new;
            float e[4];
#pragma unroll
            for (int r = 0; r < 4; ++r) e[r] = expf(s[r] - m_new);
            l_run = l_run * corr + ((e[0] + e[1]) + (e[2] + e[3]));
            u32x2 o;
            o[0] = (uint32_t)f32_to_bf16(e[0]) | ((uint32_t)f32_to_bf16(e[1]) << 16);
            o[1] = (uint32_t)f32_to_bf16(e[2]) | ((uint32_t)f32_to_bf16(e[3]) << 16);
            *(u32x2*)(ps + (hn * 16 + c) * PP + kt * 16 + 4 * g) = o;
            if (kt == 0 && g == 0) cr[hn * 16 + c] = corr;
        }
        __syncthreads();
        float corr[NH];
#pragma unroll
        for (int n = 0; n < NH; ++n) corr[n] = cr[n * 16 + c];
#pragma unroll
        for (int b = 0; b < RB; ++b) {
            const int c0 = (wave + 8 * b) * 32;
            if (c0 >= R) continue;
#pragma unroll
            for (int o = 0; o < 2; ++o)
#pragma unroll
                for (int n = 0; n < NH; ++n) acc[b][o][n] *= corr[n];
#pragma unroll
            for (int kk = 0; kk < kStep; kk += 32) {
                uint32_t x[8];
#pragma unroll
                for (int e = 0; e < 8; ++e) x[e] = *(const uint32_t*)(ks + (kk + 8 * g + e) * P + c0 + 2 * c);
                u32x4 ev, od;
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    ev[e] = __builtin_amdgcn_perm(x[2 * e + 1], x[2 * e], 0x05040100u);
                    od[e] = __builtin_amdgcn_perm(x[2 * e + 1], x[2 * e], 0x07060302u);
                }
#pragma unroll
                for (int n = 0; n < NH; ++n) {
                    const bf16x8 w = *(const bf16x8*)(ps + (n * 16 + c) * PP + kk + 8 * g);
                    acc[b][0][n] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8, ev), w, acc[b][0][n], 0, 0, 0);
                    acc[b][1][n] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8, od), w, acc[b][1][n], 0, 0, 0);
                }
            }
        }
        __syncthreads();
    }
    // ---- the record of every head: a lane holds columns 8 g .. 8 g + 7 of its blocks for head c
    if (scores) {
        l_run += lane_xor16(l_run);
        l_run += lane_xor32(l_run);
        if (g == 0) wm[kt * 16 * NH + hn * 16 + c] = l_run;
    }
    __syncthreads();
    if (scores && kt == 0 && g == 0 && head < a.heads) {
        float* rec = record(p, row, head, split);
        const int i = hn * 16 + c;
        rec[0] = m_run;
        rec[1] = (wm[i] + wm[16 * NH + i]) + (wm[32 * NH + i] + wm[48 * NH + i]);
    }
#pragma unroll
    for (int n = 0; n < NH; ++n) {
        const int h = h0 + n * 16 + c;
        if (h >= a.heads) continue;
        float* rec = record(p, row, h, split) + kRec;
#pragma unroll
        for (int b = 0; b < RB; ++b) {
            const int d = (wave + 8 * b) * 32 + 8 * g;
            if (d >= R) continue;  // (kv_rank % 8 == 0)
            const f32x4 ev = acc[b][0][n], od = acc[b][1][n];
            *(f32x4*)(rec + d) = f32x4{ev[0], od[0], ev[1], od[1]};
            *(f32x4*)(rec + d + 4) = f32x4{ev[2], od[2], ev[3], od[3]};
        }
    }
}

// ------------------------------------------------------------------------------------ splits joined, values
// weights of a (row, head)'s splits: lane = split; returns 1 / sum
__device__ __forceinline__ float split_weight(const float* rec, int ld, int n_split, int lane, float& w) {
    const bool in = lane < n_split;
    const float m = in ? rec[(int64_t)lane * ld] : -1.0e30f, l = in ? rec[(int64_t)lane * ld + 1] : 0.f;
    const float top = wave_max(m);
    w = in ? expf(m - top) : 0.f;
    return 1.0f / group_sum(w * l, 64);
}

// grid (heads, rows), 256 threads
template <typename T>
__global__ __launch_bounds__(256) void latent_out_rows_kernel(const LatParams p) {
    const mi355_latent_args& a = p.a;
    extern __shared__ __attribute__((aligned(16))) float sm[];  // [kv_rank]
    __shared__ float wgt[kMaxSplit];
    const int h = blockIdx.x, row = p.row0 + blockIdx.y, tid = threadIdx.x, lane = tid & 63;
    const float* rec = record(p, row, h, 0);
    const int ld = a.kv_rank + kRec;
    float w;
    const float inv = split_weight(rec, ld, p.n_split, lane, w);
    if (tid < p.n_split) wgt[tid] = w * inv;
    __syncthreads();
    for (int r = tid; r < a.kv_rank; r += 256) {
        float o = 0.f;
        for (int s = 0; s < p.n_split; ++s) o += wgt[s] * rec[(int64_t)s * ld + kRec + r];
        sm[r] = o;
    }
    __syncthreads();
    for (int v = tid >> 6; v < a.vdim; v += 4) {
        const T* uv = (const T*)a.uv + ((int64_t)h * a.vdim + v) * a.kv_rank;
        float s = 0.f;
        for (int r = lane; r < a.kv_rank; r += 64) s += sm[r] * to_f32<T>(uv[r]);
        s = group_sum(s, 64);
        if (lane == 0) ((T*)a.y)[(int64_t)row * a.ldy + (int64_t)h * a.vdim + v] = from_f32<T>(s);
    }
}

// grid (heads, 64-value blocks, tiles of `tile` <= 16 rows), 256 threads; kv_rank % 8 == 0, vdim % 4 == 0.  LDS: [16][pad32(kv_rank) + 8] bf16
__global__ __launch_bounds__(256) void latent_out_mfma_kernel(const LatParams p, int rows, int tile) {
    const mi355_latent_args& a = p.a;
    extern __shared__ __attribute__((aligned(16))) char smem[];
    __shared__ float wgt[16][kMaxSplit];
    const int h = blockIdx.x, t0 = p.row0 + blockIdx.z * tile, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, c = lane & 15, g = lane >> 4;
    const int end = p.row0 + rows, R = a.kv_rank, Rp = pad32(R), P = Rp + 8, ld = R + kRec;
    bf16_t* os = (bf16_t*)smem;
    const int n = min(tile, end - t0);
    for (int t = wave; t < n; t += 4) {
        float w;
        const float inv = split_weight(record(p, t0 + t, h, 0), ld, p.n_split, lane, w);
        if (lane < p.n_split) wgt[t][lane] = w * inv;
    }
    __syncthreads();
    const int quads = Rp / 4;
    for (int it = tid; it < n * quads; it += 256) {  // (rows past n: whatever stands there, in columns of the product that nobody stores)
        const int t = it / quads, r = (it - t * quads) * 4;
        f32x4 o = {0.f, 0.f, 0.f, 0.f};
        if (r < R) {
            const float* rec = record(p, t0 + t, h, 0) + kRec + r;
#pragma unroll 16
            for (int s = 0; s < p.n_split; ++s) o += wgt[t][s] * *(const f32x4*)(rec + (int64_t)s * ld);
        }
        u32x2 b;
        b[0] = (uint32_t)f32_to_bf16(o[0]) | ((uint32_t)f32_to_bf16(o[1]) << 16);
        b[1] = (uint32_t)f32_to_bf16(o[2]) | ((uint32_t)f32_to_bf16(o[3]) << 16);
        *(u32x2*)(os + t * P + r) = b;
    }
    __syncthreads();
    const int v0 = blockIdx.y * 64 + wave * 16;
    if (v0 >= a.vdim) return;
    const bf16_t* uv = (const bf16_t*)a.uv + ((int64_t)h * a.vdim + min(v0 + c, a.vdim - 1)) * R;
    f32x4 acc = {0.f, 0.f, 0.f, 0.f};
    const u32x4 zero = {0u, 0u, 0u, 0u};
    for (int d0 = 8 * g; d0 - 8 * g < Rp; d0 += 128) {
        u32x4 av[4], bv[4];
#pragma unroll
        for (int j = 0; j < 4; ++j) {
            const int d = d0 + 32 * j;
            av[j] = d < R ? *(const u32x4*)(uv + d) : zero;
            bv[j] = d < R ? *(const u32x4*)(os + c * P + d) : zero;
        }
#pragma unroll
        for (int j = 0; j < 4; ++j)
            acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8, av[j]), __builtin_bit_cast(bf16x8, bv[j]), acc, 0, 0, 0);
    }
    if (c < n && v0 + 4 * g < a.vdim) {
        u32x2 o;
        o[0] = (uint32_t)f32_to_bf16(acc[0]) | ((uint32_t)f32_to_bf16(acc[1]) << 16);
        o[1] = (uint32_t)f32_to_bf16(acc[2]) | ((uint32_t)f32_to_bf16(acc[3]) << 16);
        *(u32x2*)((bf16_t*)a.y + (int64_t)(t0 + c) * a.ldy + (int64_t)h * a.vdim + v0 + 4 * g) = o;
    }
}

// ------------------------------------------------------------------------------------ prompt steps: latents of all positions
// grid (ceil(rows_per_seq / 4), seqs), 256 threads: a wave per position; kv_rank % 8 == 0
__global__ __launch_bounds__(256) void gather_latents_kernel(const LatParams p, int ld_out) {
    const mi355_latent_args& a = p.a;
    const int seq = blockIdx.y, pos = blockIdx.x * 4 + (threadIdx.x >> 6), lane = threadIdx.x & 63;
    if (pos >= p.b.pos[seq] + p.b.count[seq]) return;
    const u32x4* src = (const u32x4*)((const bf16_t*)a.cache + ((int64_t)p.b.slot[seq] * a.cache_rows + pos) * p.ld_c);
    u32x4* dst = (u32x4*)((bf16_t*)a.rows_c + (seq * p.rows_per_seq + pos) * ld_out);
    for (int j = lane; j < ld_out / 8; j += 64) dst[j] = j < a.kv_rank / 8 ? src[j] : u32x4{0u, 0u, 0u, 0u};
}

int pad128(int n) { return (n + 127) / 128 * 128; }

bool vec_sizes(const mi355_latent_args& a) {
    return a.dtype == MI355_BF16 && a.dim % 8 == 0 && a.rot_dim % 8 == 0 && a.vdim % 8 == 0 && a.kv_rank % 8 == 0 && a.ldy % 4 == 0 &&
           (uintptr_t)a.cache % 16 == 0 && (uintptr_t)a.q % 16 == 0 && (uintptr_t)a.qa % 16 == 0 && (uintptr_t)a.uk_t % 16 == 0 &&
           (uintptr_t)a.uv % 16 == 0 && (uintptr_t)a.y % 8 == 0 && a.uq.N % 8 == 0;
}
bool mfma_fits(const mi355_latent_args& a) {
    const int dk = a.kv_rank + a.rot_dim;
    return vec_sizes(a) && a.kv_rank <= 512 && dk <= 64 * (a.kv_rank <= 256 ? kTileItems<1> : kTileItems<2>);
}
bool tiles_fit(const mi355_latent_args& a, const mi355_seq_batch& b) {
    return vec_sizes(a) && a.dim + a.rot_dim <= 256 && a.vdim <= 256 && a.expand.w && a.rows_c && a.kv_rows && b.max_end > 0 &&
           b.max_end <= a.expand_rows && (uint64_t)b.max_end * a.expand.N < 0xFFFFFFFFull && (uint64_t)b.max_end * (a.kv_rank + a.rot_dim) < 0xFFFFFFFFull &&
           (uint64_t)b.max_count * a.uq.N < 0xFFFFFFFFull && (uintptr_t)a.rows_c % 16 == 0 && (uintptr_t)a.kv_rows % 16 == 0;
}

template <int NH, int RB>
int launch_mfma(const LatParams& p, int rows, hipStream_t s) {
    const size_t lds = mfma_lds<NH>(p.a.kv_rank + p.a.rot_dim);
    static hipError_t e = hipFuncSetAttribute((const void*)latent_mfma_kernel<NH, RB>, hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024 - 64);
    MI355_CHECK_ARG(e == hipSuccess && lds <= 160 * 1024 - 64, MI355_E_SHAPE, "latent_attention: %zu bytes of LDS (%s)", lds, hipGetErrorString(e));
    hipLaunchKernelGGL((latent_mfma_kernel<NH, RB>), dim3(p.n_split, (p.a.heads + 16 * NH - 1) / (16 * NH), rows), dim3(512), lds, s, p);
    MI355_LAUNCH_CHECK();
    return 0;
}

// decode steps, short portions, f32 models: rows of the step by themselves, over the latents
template <typename T>
int run_latents(LatParams p, bool mfma, hipStream_t s) {
    const mi355_latent_args& a = p.a;
    const int rows = p.b.rows, DK = a.kv_rank + a.rot_dim;
    MI355_CHECK_ARG(a.kv_rank <= 1024 && a.dim <= 8192 && DK <= 8192, MI355_E_SHAPE, "latent_attention: latent size %d exceeds 1024", a.kv_rank);
    const int nh = a.heads > 16 ? 2 : 1;
    const int64_t groups = (int64_t)rows * (mfma ? (a.heads + 16 * nh - 1) / (16 * nh) : a.heads);
    int64_t n = (mfma ? 256 : 2048) / groups;
    n = n < a.cache_rows / 64 ? n : a.cache_rows / 64;
    n = n < kMaxSplit ? n : kMaxSplit;
    p.n_split = n < 1 ? 1 : (int)n;
    const uint64_t rec = (uint64_t)a.heads * (a.kv_rank + kRec) * 4;
    MI355_CHECK_ARG(a.partials && a.partials_bytes >= rec, MI355_E_SHAPE, "latent_attention: no room for one row's records");
    while (p.n_split > 1 && rec * p.n_split * rows > a.partials_bytes) p.n_split /= 2;
    const uint64_t fit = a.partials_bytes / (rec * p.n_split);
    const int most = fit < 65535 ? (int)fit : 65535;
    for (p.row0 = 0; p.row0 < rows; p.row0 += most) {
        const int m = rows - p.row0 < most ? rows - p.row0 : most;
        if constexpr (sizeof(T) == 2) {
            if (mfma) {
                hipLaunchKernelGGL(absorb_mfma_kernel, dim3(a.heads, (a.kv_rank + 63) / 64 + 1, (m + 15) / 16), dim3(256), 0, s, p, m);
                MI355_LAUNCH_CHECK();
                int rc;
                if (a.kv_rank <= 256) rc = nh == 2 ? launch_mfma<2, 1>(p, m, s) : launch_mfma<1, 1>(p, m, s);
                else rc = nh == 2 ? launch_mfma<2, 2>(p, m, s) : launch_mfma<1, 2>(p, m, s);
                if (rc) return rc;
                const int tile = m >= 64 ? 16 : m >= 32 ? 8 : 4;  // (the records are the bytes: enough workgroups to read them)
                hipLaunchKernelGGL(latent_out_mfma_kernel, dim3(a.heads, (a.vdim + 63) / 64, (m + tile - 1) / tile), dim3(256),
                                   (size_t)16 * (pad32(a.kv_rank) + 8) * 2, s, p, m, tile);
                MI355_LAUNCH_CHECK();
                continue;
            }
        }
        hipLaunchKernelGGL(absorb_rows_kernel<T>, dim3(a.heads, m), dim3(256), (size_t)a.dim * 4, s, p);
        MI355_LAUNCH_CHECK();
        hipLaunchKernelGGL(latent_rows_kernel<T>, dim3(p.n_split, a.heads, m), dim3(256), (size_t)(DK + 256) * 4, s, p);
        MI355_LAUNCH_CHECK();
        hipLaunchKernelGGL(latent_out_rows_kernel<T>, dim3(a.heads, m), dim3(256), (size_t)a.kv_rank * 4, s, p);
        MI355_LAUNCH_CHECK();
    }
    return 0;
}

int run_tiles(LatParams p, mi355_stream_t stream) {
    const mi355_latent_args& a = p.a;
    hipStream_t s = (hipStream_t)stream;
    const int ld_c = pad128(a.kv_rank), span = p.b.max_end;
    const int most = (int)(a.expand_rows / span);  // sequences whose positions fit the scratch together
    const mi355_seq_batch all = p.b;
    for (int s0 = 0; s0 < all.seqs; s0 += most) {
        const int n = all.seqs - s0 < most ? all.seqs - s0 : most;
        p.b.seqs = n;
        p.b.row0 = all.row0 + s0, p.b.count = all.count + s0, p.b.slot = all.slot + s0, p.b.pos = all.pos + s0;
        p.rows_per_seq = span;
        hipLaunchKernelGGL(gather_latents_kernel, dim3((span + 3) / 4, n), dim3(256), 0, s, p, ld_c);
        MI355_LAUNCH_CHECK();
        mi355_product q;
        memset(&q, 0, sizeof(q));
        q.dtype = q.y_dtype = MI355_BF16;
        q.x = a.rows_c, q.ldx = ld_c, q.M = n * span;
        q.y = a.kv_rows, q.ldy = a.expand.N, q.epi = MI355_EPI_STORE, q.alpha = 1.f;
        q.ws = a.gemm_ws, q.ws_bytes = a.gemm_ws_bytes;
        if (int rc = mi355_product_run(q, a.expand, s)) return rc;
        mi355_window_attn_args w;
        memset(&w, 0, sizeof(w));
        w.proj = a.q, w.ld = a.uq.N, w.dtype = MI355_BF16;
        w.heads = w.kv_heads = a.heads, w.dim = a.dim + a.rot_dim, w.vdim = a.vdim;
        w.off_g = -1, w.scale = a.scale, w.window = 1 << 30, w.ring = 1;
        w.rot_dims = a.rot_dim, w.rot_at = a.dim, w.inv_freq = a.inv_freq, w.sink = a.sink;
        w.y = a.y, w.ldy = a.ldy;
        w.role = MI355_KV_ROWS, w.kv_rows = a.kv_rows, w.rows_per_seq = span, w.ld_rows = a.expand.N;
        w.off_v_rows = (a.heads * a.dim + 15) / 16 * 16;
        w.tail_dims = a.rot_dim, w.key_tail = (const bf16_t*)a.cache + a.kv_rank, w.ld_tail = p.ld_c, w.tail_slot = (int64_t)a.cache_rows * p.ld_c;
        mi355_seq_batch b = p.b;
        if (int rc = mi355_window_attention(&w, &b, stream)) return rc;
    }
    return 0;
}

}  // namespace

extern "C" int mi355_latent_attention(const mi355_latent_args* a, const mi355_seq_batch* b, mi355_stream_t stream) {
    MI355_CHECK_ARG(a && b && a->proj && a->cache && a->y && a->cq && a->q && a->qa && a->q_norm && a->c_norm && a->inv_freq && a->sink && a->uq.w &&
                        a->uk_t && a->uv,
                    MI355_E_ARG, "latent_attention: null argument");
    MI355_CHECK_ARG(b->row0 && b->count && b->slot && b->pos, MI355_E_ARG, "latent_attention: null batch");
    MI355_CHECK_ARG(b->rows > 0 && b->rows <= 65535 && b->seqs > 0 && b->seqs <= b->rows && b->max_count > 0, MI355_E_SHAPE,
                    "latent_attention: bad batch (%d rows, %d sequences)", b->rows, b->seqs);
    MI355_CHECK_ARG(a->dtype == MI355_F32 || a->dtype == MI355_BF16, MI355_E_DTYPE, "latent_attention: dtype must be f32 or bf16");
    MI355_CHECK_ARG(a->heads > 0 && a->heads <= 65535 && a->dim > 0 && a->vdim > 0 && a->rot_dim >= 0 && a->rot_dim % 2 == 0 && a->q_rank > 0 &&
                        a->kv_rank > 0 && a->cache_rows > 0 && a->uq.K == a->q_rank && a->uq.N >= a->heads * (a->dim + a->rot_dim),
                    MI355_E_SHAPE, "latent_attention: bad sizes (heads %d, %d + %d, values %d, ranks %d / %d)", a->heads, a->dim, a->rot_dim, a->vdim,
                    a->q_rank, a->kv_rank);
    hipStream_t s = (hipStream_t)stream;
    LatParams p;
    p.a = *a;
    p.b = *b;
    p.fresh = b->max_count == 1;
    p.row0 = 0;
    p.n_split = 1;
    p.ld_c = a->kv_rank + a->rot_dim;
    p.ld_cq = pad128(a->q_rank);
    p.ld_qh = a->dim + a->rot_dim;
    p.rows_per_seq = 0;
    const bool f32 = a->dtype == MI355_F32;
    const bool vec = vec_sizes(*a) && a->q_rank % 8 == 0 && a->ld % 8 == 0 && a->off_q % 8 == 0 && a->off_c % 8 == 0 && (uintptr_t)a->proj % 16 == 0 &&
                     (uintptr_t)a->cq % 16 == 0;
    if (f32) hipLaunchKernelGGL((latent_prep_kernel<float, 1>), dim3(b->rows), dim3(256), 0, s, p);
    else if (vec) hipLaunchKernelGGL((latent_prep_kernel<bf16_t, 8>), dim3(b->rows), dim3(256), 0, s, p);
    else hipLaunchKernelGGL((latent_prep_kernel<bf16_t, 1>), dim3(b->rows), dim3(256), 0, s, p);
    MI355_LAUNCH_CHECK();
    mi355_product q;
    memset(&q, 0, sizeof(q));
    q.dtype = q.y_dtype = a->dtype;
    q.x = a->cq, q.ldx = p.ld_cq, q.M = b->rows;
    q.y = a->q, q.ldy = a->uq.N, q.epi = MI355_EPI_STORE, q.alpha = 1.f;
    q.ws = a->gemm_ws, q.ws_bytes = a->gemm_ws_bytes;
    if (int rc = mi355_product_run(q, a->uq, s)) return rc;
    const bool tiles = !p.fresh && tiles_fit(*a, *b), mfma = mfma_fits(*a);
    MI355_CHECK_ARG((a->path != 2 || mfma) && (a->path != 3 || tiles), MI355_E_SHAPE, "latent_attention: this shape does not take path %d", a->path);
    // (a handful of rows per sequence would leave most of a 128-query tile empty)
    if (a->path == 3 || (a->path == 0 && tiles && b->max_count > 8)) return run_tiles(p, stream);
    return f32 ? run_latents<float>(p, false, s) : run_latents<bf16_t>(p, mfma && a->path != 1, s);
}
