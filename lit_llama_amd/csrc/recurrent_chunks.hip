// Prompt steps of the linear recurrences in chunks of 64 rows, on the f32 matrix cores (v_mfma_f32_16x16x4_f32: operands, products and
// sums are f32, as the recurrence asks).
//
// With G_i = sum of the log decays of a chunk up to row i, S_0 the state in front of the chunk and U the rows written into it:
//
//   delta  (I + A) U = diag(beta) (V - diag(e^G) K S_0),   A_ij = beta_i e^(G_i - G_j) k_i . k_j  (j < i)
//          O = diag(e^G) Q S_0 + P U,                      P_ij = e^(G_i - G_j) q_i . k_j         (j <= i)
//          S = e^(G_end) S_0 + K^T diag(e^(G_end - G)) U
//   gla    U = V,  e^(G_i - G_j) acts per key channel inside the products,  O = (Q e^G) S_0 + P V,  S = diag(e^(G_end)) S_0 + (K e^(G_end - G))^T V
//   ssd    as delta with U = V and A = 0 (no unit norms):  P_ij = e^(G_i - G_j) dt_j q_i . k_j (+ skip on the diagonal),
//          S = e^(G_end) S_0 + K^T diag(e^(G_end - G) dt) V
//   wkv    as gla, but row i reads the state in front of it: e^(G_(i-1) - G_j) and Q e^(G_(i-1)), and P_ii = sum q_i u k_i
//
// Every exponent is <= 0.  Launches of a step (each over all chunks at once but the scan):
//   delta_qk_kernel    delta, ssd: convolutions, unit norms (delta); Q, K^T, K K^T (delta), Q K^T per key head
//   delta_head_kernel  decays, T = (I + A)^-1 by 16 x 16 blocks, U0 = T diag(beta) V, W = T diag(beta e^G) K, P per head
//   ssd_head_kernel    decays, V^T with its convolution, P per head
//   gla_prep_kernel    gla, wkv: decays, Q e^G, (K e^(G_end - G))^T, P (off-diagonal 16 x 16 blocks anchored at the row block's first row), V^T
//   scan_kernel        one workgroup per (sequence, head, 16 columns): U = U0 - W S_0, S; the state in accumulator registers
//   chunk_out_kernel   O, output norm, gate
//
// Matrix operand layouts: A row-major and B column-major in memory with the contraction index contiguous; of every 16 of it lane group g
// (lane >> 4) takes 4g .. 4g + 3 with one 16-B load, one element per MFMA.
#include "recurrent.h"

namespace {

constexpr int kC = 64;        // rows of a chunk
constexpr int kP = kC + 4;    // pitch of [..][64] matrices in LDS
constexpr int kX = 20;        // pitch of [..][16] ones

__device__ __forceinline__ f32x4 mfma4(f32x4 a, f32x4 b, f32x4 c) {
#pragma unroll
    for (int j = 0; j < 4; ++j) c = __builtin_amdgcn_mfma_f32_16x16x4f32(a[j], b[j], c, 0, 0, 0);
    return c;
}
__device__ __forceinline__ f32x4 zero4() { return f32x4{0.f, 0.f, 0.f, 0.f}; }

// a barrier for data in LDS: global requests stay in flight across it
__device__ __forceinline__ void lds_barrier() {
    asm volatile("s_waitcnt lgkmcnt(0)\n\ts_barrier" ::: "memory");
}

// ---------------------------------------------------------------- scratch, per packed chunk (padded sizes DP, VP: multiples of 16)
struct Scratch {
    float* q;     // [NC][GQ][64][DP]        delta: unit q * q_scale; ssd: q; gla: q e^G * q_scale
    float* kt;    // [NC][GQ][DP][64]        delta: unit k; ssd: k; gla: k e^(G_end - G)
    float* kk;    // [NC][G][64][64]         delta: k_i . k_j
    float* qk;    // [NC][G][64][64]         delta, ssd: q_i . k_j
    float* P;     // [NC][H][64][64]
    float* W;     // [NC][H][64][DP]         delta
    float* ut;    // [NC][H][VP][64]         U^T (delta: U0^T until the scan)
    float* st;    // [NC][H][VP][DP]         S_0^T
    float* gam;   // [NC][H][DP]             e^(G_end) (delta, ssd: element 0)
    float* eg;    // [NC][H][64]             delta, ssd: e^G
    float* ed;    // [NC][H][64]             delta: e^(G_end - G); ssd: e^(G_end - G) dt
};

struct ChunkParams {
    RecParams r;
    Scratch s;
    int seq0;     // first sequence of this group
    int GQ, DP, VP;
};

__device__ __forceinline__ int chunk_base(const ChunkParams& p, int seq) {
    return p.r.b.row0[seq] / kC + seq - (p.r.b.row0[p.seq0] / kC + p.seq0);
}

// launches over (chunk, head): grid (8 * ceil(heads / 8) * chunks, seqs), a head's chunks on one XCD (block index mod 8), as its scan
__device__ __forceinline__ bool head_chunk(const ChunkParams& p, int& head, int& chunk) {
    const int chunks = (p.r.b.max_count + kC - 1) / kC, idx = blockIdx.x >> 3;
    head = (blockIdx.x & 7) + 8 * (idx / chunks);
    chunk = idx % chunks;
    return head < p.r.a.heads;
}

// ------------------------------------------------------------------------------------ delta, ssd: q, k per key head
// grid (chunks, kv_heads, seqs), 256 threads.  LDS: k, q [64][DP + 4]
template <typename T, int KIND>
__global__ __launch_bounds__(256) void delta_qk_kernel(const ChunkParams p) {
    const mi355_recurrent_args& a = p.r.a;
    extern __shared__ __attribute__((aligned(16))) float sm[];
    const int seq = p.seq0 + blockIdx.z, kvh = blockIdx.y, t0 = blockIdx.x * kC;
    const int cnt = p.r.b.count[seq];
    if (t0 >= cnt) return;
    const int DP = p.DP, ld = DP + 4, dim = a.dim;
    float* k = sm;
    float* q = sm + kC * ld;
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int pos0 = p.r.b.pos[seq];
    const T* rows = (const T*)a.proj + (int64_t)p.r.b.row0[seq] * a.ld;
    const int ring_ld = 2 * a.kv_heads * dim + a.heads * a.vdim;
    const T* ring = (const T*)a.conv_ring + (int64_t)p.r.b.slot[seq] * a.taps * ring_ld;
    for (int i = tid; i < 8 * DP; i += 256) {  // (q or k, 16-row block, channel)
        const int d = i % DP, blk = i / DP, t = (blk & 3) * 16, is_k = blk >> 2;
        float y[16];
        if (d < dim) {
            const int c = kvh * dim + d;
            conv_rows16<T>(a, rows, ring, ring_ld, (is_k ? a.off_k : a.off_q) + c, is_k * a.kv_heads * dim + c,
                           (is_k ? a.conv_k : a.conv_q) + (int64_t)c * a.taps, t0 + t, cnt, pos0, y,
                           KIND == MI355_REC_SSD ? conv_bias(is_k ? a.conv_bk : a.conv_bq, c) : 0.f);
        } else {
#pragma unroll
            for (int e = 0; e < 16; ++e) y[e] = 0.f;
        }
        float* dst = (is_k ? k : q) + t * ld + d;
#pragma unroll
        for (int e = 0; e < 16; ++e) dst[e * ld] = y[e];
    }
    __syncthreads();
    for (int t = KIND == MI355_REC_DELTA ? wave : kC; t < kC; t += 4) {  // unit vectors: a wave per row
        float sq = 0.f, sk = 0.f;
        for (int d = lane; d < dim; d += 64) {
            sq += q[t * ld + d] * q[t * ld + d];
            sk += k[t * ld + d] * k[t * ld + d];
        }
        sq = group_sum(sq, 64);
        sk = group_sum(sk, 64);
        const float iq = a.q_scale / sqrtf(sq + a.unit_eps), ik = 1.0f / sqrtf(sk + a.unit_eps);
        for (int d = lane; d < dim; d += 64) {
            q[t * ld + d] *= iq;
            k[t * ld + d] *= ik;
        }
    }
    __syncthreads();
    const int64_t gi = (int64_t)(chunk_base(p, seq) + blockIdx.x) * p.GQ + kvh;
    float* oq = p.s.q + gi * kC * DP;
    float* okt = p.s.kt + gi * DP * kC;
    for (int i = tid; i < kC * DP / 4; i += 256) {
        const int t = i / (DP / 4), d = (i - t * (DP / 4)) * 4;
        *(f32x4*)(oq + t * DP + d) = *(const f32x4*)(q + t * ld + d);
    }
    for (int i = tid; i < kC * DP / 4; i += 256) {
        const int d = i / (kC / 4), t = (i - d * (kC / 4)) * 4;
        *(f32x4*)(okt + d * kC + t) = f32x4{k[t * ld + d], k[(t + 1) * ld + d], k[(t + 2) * ld + d], k[(t + 3) * ld + d]};
    }
    // wave w: rows 16 w .. 16 w + 15 of K K^T and Q K^T, column blocks up to its own
    const int c16 = lane & 15, g = lane >> 4;
    float* okk = p.s.kk + gi * kC * kC;
    float* oqk = p.s.qk + gi * kC * kC;
    for (int cb = 0; cb <= wave; ++cb) {
        f32x4 akk = zero4(), aqk = zero4();
        for (int d = 4 * g; d < DP; d += 16) {
            const f32x4 b = *(const f32x4*)(k + (cb * 16 + c16) * ld + d);
            if constexpr (KIND == MI355_REC_DELTA) akk = mfma4(*(const f32x4*)(k + (wave * 16 + c16) * ld + d), b, akk);
            aqk = mfma4(*(const f32x4*)(q + (wave * 16 + c16) * ld + d), b, aqk);
        }
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            if constexpr (KIND == MI355_REC_DELTA) okk[(wave * 16 + 4 * g + r) * kC + cb * 16 + c16] = akk[r];
            oqk[(wave * 16 + 4 * g + r) * kC + cb * 16 + c16] = aqk[r];
        }
    }
}

// ------------------------------------------------------------------------------------ delta: per head
// 256 threads.  LDS: A, T [64][kP], X [64][kX], vt [VP][kP]
template <typename T>
__global__ __launch_bounds__(256) void delta_head_kernel(const ChunkParams p) {
    const mi355_recurrent_args& a = p.r.a;
    extern __shared__ __attribute__((aligned(16))) float sm[];
    __shared__ double gcum[kC];
    __shared__ float beta[kC], bg[kC];
    int head, chunk;
    if (!head_chunk(p, head, chunk)) return;
    const int seq = p.seq0 + blockIdx.y, t0 = chunk * kC;
    const int cnt = p.r.b.count[seq];
    if (t0 >= cnt) return;
    const int DP = p.DP, VP = p.VP;
    float* A = sm;
    float* Ti = A + kC * kP;
    float* X = Ti + kC * kP;
    float* vt = X + kC * kX;
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int c16 = lane & 15, g = lane >> 4;
    const int kvh = head / (a.heads / a.kv_heads);
    const int pos0 = p.r.b.pos[seq];
    const T* rows = (const T*)a.proj + (int64_t)p.r.b.row0[seq] * a.ld;
    const int ring_ld = 2 * a.kv_heads * a.dim + a.heads * a.vdim;
    const T* ring = (const T*)a.conv_ring + (int64_t)p.r.b.slot[seq] * a.taps * ring_ld;
    const int64_t ci = chunk_base(p, seq) + chunk;
    const int64_t gi = ci * p.GQ + kvh, hi = ci * a.heads + head;

    if (tid < kC) {
        float lg = 0.f, b = 0.f;
        if (t0 + tid < cnt) {
            const T* row = rows + (int64_t)(t0 + tid) * a.ld;
            lg = -expf(a.a_log[head]) * softplus_f32(to_f32<T>(row[a.off_a + head]) + a.dt_bias[head]);
            b = sigmoid_f32(to_f32<T>(row[a.off_b + head]));
        }
        // inclusive sum over the wave; f64, so that differences of far sums keep f32 accuracy
        double s = lg;
#pragma unroll
        for (int o = 1; o < 64; o <<= 1) {
            const double v = __shfl_up(s, o, 64);
            if (lane >= o) s += v;
        }
        gcum[tid] = s;
        beta[tid] = b;
        const double end = __shfl(s, 63, 64);
        const float eg = expf((float)s);
        bg[tid] = b * eg;
        p.s.eg[hi * kC + tid] = eg;
        p.s.ed[hi * kC + tid] = expf((float)(end - s));
        if (tid == 63) p.s.gam[hi * DP] = expf((float)end);
    }
    // V^T with the convolution (beta rides on it below)
    for (int i = tid; i < 4 * VP; i += 256) {
        const int d = i % VP, t = (i / VP) * 16;
        float y[16];
        if (d < a.vdim) {
            const int c = head * a.vdim + d;
            conv_rows16<T>(a, rows, ring, ring_ld, a.off_v + c, 2 * a.kv_heads * a.dim + c, a.conv_v + (int64_t)c * a.taps, t0 + t, cnt, pos0, y);
        } else {
#pragma unroll
            for (int e = 0; e < 16; ++e) y[e] = 0.f;
        }
#pragma unroll
        for (int e = 0; e < 4; ++e) *(f32x4*)(vt + d * kP + t + 4 * e) = f32x4{y[4 * e], y[4 * e + 1], y[4 * e + 2], y[4 * e + 3]};
    }
    __syncthreads();
    const float* kk = p.s.kk + gi * kC * kC;
    const float* qk = p.s.qk + gi * kC * kC;
    float* oP = p.s.P + hi * kC * kC;
#pragma unroll 8
    for (int n = 0; n < kC * kC / 256; ++n) {
        const int i = n * 256 + tid, r = i >> 6, c = i & 63;
        const float qv = qk[i], kv = kk[i];  // (above the diagonal blocks: unwritten scratch, dropped below)
        const float e = c <= r ? exp_f32((float)(gcum[r] - gcum[c])) : 0.f;
        A[r * kP + c] = c < r ? beta[r] * e * kv : 0.f;
        Ti[r * kP + c] = 0.f;
        oP[i] = c <= r ? e * qv : 0.f;
    }
    for (int i = tid; i < kC * VP; i += 256) {
        const int d = i / kC, t = i - d * kC;
        vt[d * kP + t] *= beta[t];
    }
    __syncthreads();
    // ---- diagonal blocks of T: thread (block, column), forward substitution in registers
    if (tid < 64) {
        const int b0 = (tid >> 4) * 16, c = tid & 15;
        float x[16];
#pragma unroll
        for (int i = 0; i < 16; ++i) {
            float s = i == c ? 1.f : 0.f;
#pragma unroll
            for (int j = 0; j < i; ++j) s -= A[(b0 + i) * kP + b0 + j] * x[j];
            x[i] = i < c ? 0.f : s;
        }
#pragma unroll
        for (int i = 0; i < 16; ++i) Ti[(b0 + i) * kP + b0 + c] = x[i];
    }
    __syncthreads();
    // ---- below the diagonal, distance by distance: T_ij = -T_ii sum_{j <= k < i} A_ik T_kj; wave j takes column block j.
    // X holds the transposed sum (the B operand of the second product); T_kj is read as B from row-major T
    for (int dist = 1; dist < 4; ++dist) {
        const int jb = wave, ib = jb + dist;
        if (ib < 4) {
            f32x4 s = zero4();
            for (int kb = jb; kb < ib; ++kb) {
                const f32x4 av = *(const f32x4*)(A + (ib * 16 + c16) * kP + kb * 16 + 4 * g);
                f32x4 bv;
#pragma unroll
                for (int j = 0; j < 4; ++j) bv[j] = Ti[(kb * 16 + 4 * g + j) * kP + jb * 16 + c16];
                s = mfma4(av, bv, s);
            }
            // D: rows 4 g + r, column c16 -> X[column][row]
            *(f32x4*)(X + (jb * 16 + c16) * kX + 4 * g) = s;
        }
        __syncthreads();
        if (ib < 4) {
            const f32x4 av = *(const f32x4*)(Ti + (ib * 16 + c16) * kP + ib * 16 + 4 * g);
            const f32x4 bv = *(const f32x4*)(X + (jb * 16 + c16) * kX + 4 * g);
            const f32x4 t = mfma4(av, bv, zero4());
#pragma unroll
            for (int r = 0; r < 4; ++r) Ti[(ib * 16 + 4 * g + r) * kP + jb * 16 + c16] = -t[r];
        }
        __syncthreads();
    }
    // ---- U0^T and W: wave w holds rows 16 w .. 16 w + 15 (T is lower triangular: columns up to 16 w + 15)
    f32x4 ta[4];
#pragma unroll
    for (int kb = 0; kb < 4; ++kb) ta[kb] = *(const f32x4*)(Ti + (wave * 16 + c16) * kP + kb * 16 + 4 * g);
    float* out = p.s.ut + hi * VP * kC;
    for (int nb = 0; nb < VP / 16; ++nb) {
        f32x4 acc = zero4();
#pragma unroll
        for (int kb = 0; kb < 4; ++kb)
            if (kb <= wave) acc = mfma4(ta[kb], *(const f32x4*)(vt + (nb * 16 + c16) * kP + kb * 16 + 4 * g), acc);
        *(f32x4*)(out + (nb * 16 + c16) * kC + wave * 16 + 4 * g) = acc;
    }
    const float* kt = p.s.kt + gi * DP * kC;
    float* oW = p.s.W + hi * kC * DP;
    f32x4 bgv[4];
#pragma unroll
    for (int kb = 0; kb < 4; ++kb) bgv[kb] = *(const f32x4*)(bg + kb * 16 + 4 * g);
    for (int nb = 0; nb < DP / 16; ++nb) {
        f32x4 acc = zero4();
#pragma unroll
        for (int kb = 0; kb < 4; ++kb)
            if (kb <= wave) acc = mfma4(ta[kb], *(const f32x4*)(kt + (nb * 16 + c16) * kC + kb * 16 + 4 * g) * bgv[kb], acc);
#pragma unroll
        for (int r = 0; r < 4; ++r) oW[(wave * 16 + 4 * g + r) * DP + nb * 16 + c16] = acc[r];
    }
}

// ------------------------------------------------------------------------------------ ssd: per head
// 256 threads
template <typename T>
__global__ __launch_bounds__(256) void ssd_head_kernel(const ChunkParams p) {
    const mi355_recurrent_args& a = p.r.a;
    __shared__ double gcum[kC];
    __shared__ float step[kC];
    int head, chunk;
    if (!head_chunk(p, head, chunk)) return;
    const int seq = p.seq0 + blockIdx.y, t0 = chunk * kC;
    const int cnt = p.r.b.count[seq];
    if (t0 >= cnt) return;
    const int DP = p.DP, VP = p.VP, tid = threadIdx.x, lane = tid & 63;
    const int kvh = head / (a.heads / a.kv_heads);
    const int pos0 = p.r.b.pos[seq];
    const T* rows = (const T*)a.proj + (int64_t)p.r.b.row0[seq] * a.ld;
    const int ring_ld = 2 * a.kv_heads * a.dim + a.heads * a.vdim;
    const T* ring = (const T*)a.conv_ring + (int64_t)p.r.b.slot[seq] * a.taps * ring_ld;
    const int64_t ci = chunk_base(p, seq) + chunk;
    const int64_t gi = ci * p.GQ + kvh, hi = ci * a.heads + head;
    if (tid < kC) {
        float dt = 0.f, lg = 0.f;
        if (t0 + tid < cnt) {
            dt = softplus_f32(to_f32<T>(rows[(int64_t)(t0 + tid) * a.ld + a.off_a + head]) + a.dt_bias[head]);
            lg = -expf(a.a_log[head]) * dt;
        }
        double s = lg;  // inclusive sum over the wave; f64, so that differences of far sums keep f32 accuracy
#pragma unroll
        for (int o = 1; o < 64; o <<= 1) {
            const double v = __shfl_up(s, o, 64);
            if (lane >= o) s += v;
        }
        gcum[tid] = s;
        step[tid] = dt;
        const double end = __shfl(s, 63, 64);
        p.s.eg[hi * kC + tid] = expf((float)s);
        p.s.ed[hi * kC + tid] = expf((float)(end - s)) * dt;
        if (tid == 63) p.s.gam[hi * DP] = expf((float)end);
    }
    float* out = p.s.ut + hi * VP * kC;
    for (int i = tid; i < 4 * VP; i += 256) {
        const int d = i % VP, t = (i / VP) * 16;
        float y[16];
        if (d < a.vdim) {
            const int c = head * a.vdim + d;
            conv_rows16<T>(a, rows, ring, ring_ld, a.off_v + c, 2 * a.kv_heads * a.dim + c, a.conv_v + (int64_t)c * a.taps, t0 + t, cnt, pos0, y,
                           conv_bias(a.conv_bv, c));
        } else {
#pragma unroll
            for (int e = 0; e < 16; ++e) y[e] = 0.f;
        }
#pragma unroll
        for (int e = 0; e < 4; ++e) *(f32x4*)(out + d * kC + t + 4 * e) = f32x4{y[4 * e], y[4 * e + 1], y[4 * e + 2], y[4 * e + 3]};
    }
    __syncthreads();
    const float* qk = p.s.qk + gi * kC * kC;
    float* oP = p.s.P + hi * kC * kC;
    const float skip = a.skip[head];
#pragma unroll 8
    for (int n = 0; n < kC * kC / 256; ++n) {
        const int i = n * 256 + tid, r = i >> 6, c = i & 63;
        const float qv = qk[i];  // (above the diagonal blocks: unwritten scratch, dropped)
        oP[i] = c <= r ? exp_f32((float)(gcum[r] - gcum[c])) * step[c] * qv + (c == r ? skip : 0.f) : 0.f;
    }
}

// ------------------------------------------------------------------------------------ gla, wkv: per head
// 256 threads; key channels in slices of 64.  LDS: q, k, G [64 rows][68], low-rank rows [64][rank], sums
constexpr int kCh = 64;
template <typename T, int KIND>
__global__ __launch_bounds__(256) void gla_prep_kernel(const ChunkParams p) {
    const mi355_recurrent_args& a = p.r.a;
    extern __shared__ __attribute__((aligned(16))) float sm[];
    int head, chunk;
    if (!head_chunk(p, head, chunk)) return;
    const int seq = p.seq0 + blockIdx.y, t0 = chunk * kC;
    const int cnt = p.r.b.count[seq];
    if (t0 >= cnt) return;
    const int DP = p.DP, VP = p.VP, dim = a.dim, rank = a.rank;
    float* q = sm;
    float* k = q + kC * kP;
    float* G = k + kC * kP;
    float* seg = G + kC * kP;       // [4][64]
    float* us = seg + 4 * kCh;      // [64] wkv: bonus
    float* lr = us + kCh;           // [rank][64]
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int c16 = lane & 15, g = lane >> 4;
    const T* rows = (const T*)a.proj + (int64_t)(p.r.b.row0[seq] + t0) * a.ld;
    const int n = min(kC, cnt - t0);
    const int64_t hi = (int64_t)(chunk_base(p, seq) + chunk) * a.heads + head;
    for (int i = tid; i < kC * rank; i += 256) {
        const int t = i / rank, r = i - t * rank;
        const float lv = t < n ? to_f32<T>(rows[(int64_t)t * a.ld + a.off_a + r]) : 0.f;
        lr[r * kC + t] = KIND == MI355_REC_WKV ? tanhf(lv) : lv;
    }
    float* oq = p.s.q + hi * kC * DP;
    float* okt = p.s.kt + hi * DP * kC;
    f32x4 off[4];                    // wave w: P blocks (w, 0 .. w - 1)
#pragma unroll
    for (int i = 0; i < 4; ++i) off[i] = zero4();
    float dg[4] = {0.f, 0.f, 0.f, 0.f};  // wave w: rows 4 rr + g of diagonal block w, column c16
    for (int c0 = 0; c0 < DP; c0 += kCh) {
        __syncthreads();
        // ---- decays: thread = (channel, 16-row block)
        {
            const int c = tid & 63, sb = tid >> 6, ch = c0 + c;
            const bool ok = ch < dim;
            T qv[16], kv[16];
            float z[16];
#pragma unroll
            for (int e = 0; e < 16; ++e) {  // (all requests first: no branches)
                const T* row = rows + (int64_t)min(sb * 16 + e, n - 1) * a.ld + head * dim + (ok ? ch : 0);
                qv[e] = row[a.off_q];
                kv[e] = row[a.off_k];
            }
            const float* w = a.a2 + (int64_t)(head * dim + (ok ? ch : 0)) * rank;
            const float bias = ok ? a.a2_bias[head * dim + ch] : 0.f;
#pragma unroll
            for (int e = 0; e < 16; ++e) z[e] = bias;
#pragma unroll 4
            for (int r = 0; r < rank; ++r) {
                const float wr = w[r];
#pragma unroll
                for (int e = 0; e < 16; e += 4) {
                    const f32x4 l = *(const f32x4*)(lr + r * kC + sb * 16 + e);
#pragma unroll
                    for (int j = 0; j < 4; ++j) z[e + j] += wr * l[j];
                }
            }
            float s = 0.f;
#pragma unroll
            for (int e = 0; e < 16; ++e) {
                const int t = sb * 16 + e;
                s += !(ok && t < n) ? 0.f : KIND == MI355_REC_WKV ? wkv_log_decay(z[e]) : -softplus_f32(-z[e]) * a.inv_tau;
                G[t * kP + c] = s;   // sums from the block's first row on
                q[t * kP + c] = ok && t < n ? to_f32<T>(qv[e]) * a.q_scale : 0.f;
                k[t * kP + c] = ok && t < n ? to_f32<T>(kv[e]) : 0.f;
            }
            seg[sb * kCh + c] = s;
            if constexpr (KIND == MI355_REC_WKV) {
                if (sb == 0) us[c] = ok ? a.bonus[head * dim + ch] : 0.f;
            }
        }
        __syncthreads();
        // what row i's query sees of the decays since its block's first row: up to its own row, or (wkv) to the row in front of it
        auto q_sum = [&](int i, int c) {
            if constexpr (KIND == MI355_REC_WKV) return (i & 15) == 0 ? zero4() : *(const f32x4*)(G + (i - 1) * kP + c);
            return *(const f32x4*)(G + i * kP + c);
        };
        // ---- diagonal blocks: wave = block, lane group g and c16 = column j, rows 4 rr + g
#pragma unroll 2
        for (int c = 0; c < kCh; c += 4) {
            const int j = wave * 16 + c16;
            const f32x4 kj = *(const f32x4*)(k + j * kP + c), gj = *(const f32x4*)(G + j * kP + c);
#pragma unroll
            for (int rr = 0; rr < 4; ++rr) {
                const int i = wave * 16 + rr * 4 + g;
                const f32x4 qi = *(const f32x4*)(q + i * kP + c), gi = q_sum(i, c);
                if constexpr (KIND == MI355_REC_WKV) {
                    const bool own = i == j;
                    const f32x4 u4 = *(const f32x4*)(us + c);
#pragma unroll
                    for (int e = 0; e < 4; ++e) dg[rr] += qi[e] * kj[e] * (own ? u4[e] : exp_f32(fminf(gi[e] - gj[e], 0.f)));
                } else {
#pragma unroll
                    for (int e = 0; e < 4; ++e) dg[rr] += qi[e] * kj[e] * exp_f32(fminf(gi[e] - gj[e], 0.f));  // (j > i: dropped at the end)
                }
            }
        }
        // ---- off-diagonal blocks (I, J): q_i e^(G_i - start of I) against k_j e^(start of I - G_j)
        for (int J = 0; J < wave; ++J)
            for (int cb = 0; cb < kCh; cb += 16) {
                const int c = cb + 4 * g;
                const int i = wave * 16 + c16, j = J * 16 + c16;
                f32x4 gap = *(const f32x4*)(seg + J * kCh + c) - *(const f32x4*)(G + j * kP + c);  // from j to the end of block J
                for (int m = J + 1; m < wave; ++m) gap += *(const f32x4*)(seg + m * kCh + c);
                f32x4 av = *(const f32x4*)(q + i * kP + c), bv = *(const f32x4*)(k + j * kP + c);
                const f32x4 gi = q_sum(i, c);
#pragma unroll
                for (int e = 0; e < 4; ++e) {
                    av[e] *= exp_f32(gi[e]);
                    bv[e] *= exp_f32(gap[e]);
                }
#pragma unroll
                for (int b = 0; b < 3; ++b)  // (constant register index)
                    if (b == J) off[b] = mfma4(av, bv, off[b]);
            }
        // ---- q e^G and (k e^(G_end - G))^T of the slice
        const int nch = min(kCh, DP - c0);
        {   // wave = 16-row block, lane = channel
            const int c = lane;
            float before = 0.f;
            for (int m = 0; m < wave; ++m) before += seg[m * kCh + c];
            if (c < nch) {
#pragma unroll
                for (int e = 0; e < 16; ++e) {
                    const int t = wave * 16 + e;
                    const float own = KIND == MI355_REC_WKV ? (e == 0 ? 0.f : G[(t - 1) * kP + c]) : G[t * kP + c];
                    oq[t * DP + c0 + c] = q[t * kP + c] * exp_f32(before + own);
                }
            }
        }
        {   // thread = (4 rows, channel c4 + 16 e)
            const int t = (tid & 15) * 4, sb = t >> 4;
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                const int c = (tid >> 4) + 16 * e;
                float rest = 0.f;
#pragma unroll
                for (int m = 0; m < 4; ++m) rest += m >= sb ? seg[m * kCh + c] : 0.f;
                f32x4 o;
#pragma unroll
                for (int j = 0; j < 4; ++j) o[j] = k[(t + j) * kP + c] * exp_f32(rest - G[(t + j) * kP + c]);
                if (c < nch) *(f32x4*)(okt + (c0 + c) * kC + t) = o;
            }
        }
        if (tid < nch) p.s.gam[hi * DP + c0 + tid] = expf(seg[tid] + seg[kCh + tid] + seg[2 * kCh + tid] + seg[3 * kCh + tid]);
    }
    float* oP = p.s.P + hi * kC * kC;
#pragma unroll
    for (int rr = 0; rr < 4; ++rr) oP[(wave * 16 + rr * 4 + g) * kC + wave * 16 + c16] = c16 <= rr * 4 + g ? dg[rr] : 0.f;
#pragma unroll
    for (int J = 0; J < 3; ++J)
        if (J < wave) {
#pragma unroll
            for (int r = 0; r < 4; ++r) oP[(wave * 16 + 4 * g + r) * kC + J * 16 + c16] = off[J][r];
        }
    for (int i = lane; i < 16 * (3 - wave) * 16; i += 64) {  // above the diagonal: zeros
        const int w = (3 - wave) * 16, r = i / w;
        oP[(wave * 16 + r) * kC + (wave + 1) * 16 + (i - r * w)] = 0.f;
    }
    float* out = p.s.ut + hi * VP * kC;
    for (int i = tid; i < kC * VP; i += 256) {
        const int d = i >> 6, t = i & 63;
        out[i] = d < a.vdim && t < n ? to_f32<T>(rows[(int64_t)t * a.ld + a.off_v + head * a.vdim + d]) : 0.f;
    }
}

// ------------------------------------------------------------------------------------ the serial part
// grid (8 * ceil(heads / 8) * VP / 16, seqs), 256 threads; NT = 16-row tiles of the state per wave (DP <= 64 NT).  The column slices of
// a head run on one XCD (block index mod 8): its L2 then serves W and K^T to all of them
template <int KIND, int NT>
__global__ __launch_bounds__(256) void scan_kernel(const ChunkParams p) {
    const mi355_recurrent_args& a = p.r.a;
    extern __shared__ __attribute__((aligned(16))) float sm[];
    const int DP = p.DP, VP = p.VP, ls = DP + 4;
    const int slices = VP / 16, idx = blockIdx.x >> 3;
    const int seq = p.seq0 + blockIdx.y, head = (blockIdx.x & 7) + 8 * (idx / slices), n0 = (idx % slices) * 16;
    if (head >= a.heads) return;
    float* sl = sm;            // [16][DP + 4]: S_0 columns
    float* ul = sm + 16 * ls;  // [16][kP]: U columns, weighted by e^(G_end - G)
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int c16 = lane & 15, g = lane >> 4;
    const int n_chunks = (p.r.b.count[seq] + kC - 1) / kC;
    constexpr bool kScalar = has_conv(KIND);  // one decay per head
    const int kvh = kScalar ? head / (a.heads / a.kv_heads) : head;
    float* state = a.state + ((int64_t)p.r.b.slot[seq] * a.heads + head) * a.dim * a.vdim;
    const int64_t cb = chunk_base(p, seq);
    const int n_tiles = DP / 16;
    const bool col_ok = n0 + c16 < a.vdim;

    f32x4 S[NT];
#pragma unroll
    for (int t = 0; t < NT; ++t)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const int i = (wave + 4 * t) * 16 + 4 * g + r;
            S[t][r] = (col_ok && i < a.dim) ? state[(int64_t)i * a.vdim + n0 + c16] : 0.f;
        }
    // a chunk's operands of this wave: two sets, the next chunk's requested when a chunk begins
    struct Ops {
        f32x4 w[KIND == MI355_REC_DELTA ? 4 * NT : 1], k[NT][4], u, d, g[NT], v[4], e[KIND == MI355_REC_SSD ? 4 : 1];
    };
    auto load = [&](int ch, Ops& x) {
        const int64_t hi = (cb + ch) * a.heads + head, gi = (cb + ch) * p.GQ + kvh;
        const float* ut = p.s.ut + hi * VP * kC + (int64_t)(n0 + c16) * kC;
        if constexpr (KIND == MI355_REC_DELTA) {
            const float* W = p.s.W + hi * kC * DP + (int64_t)(wave * 16 + c16) * DP;
#pragma unroll
            for (int b = 0; b < 4 * NT; ++b) x.w[b] = *(const f32x4*)(W + min(b, n_tiles - 1) * 16 + 4 * g);
            x.u = *(const f32x4*)(ut + wave * 16 + 4 * g);
            x.d = *(const f32x4*)(p.s.ed + hi * kC + wave * 16 + 4 * g);
            const float gm = p.s.gam[hi * DP];
            x.g[0] = f32x4{gm, gm, gm, gm};
        } else if constexpr (KIND == MI355_REC_SSD) {
#pragma unroll
            for (int b = 0; b < 4; ++b) x.v[b] = *(const f32x4*)(ut + b * 16 + 4 * g);
#pragma unroll
            for (int b = 0; b < 4; ++b) x.e[b] = *(const f32x4*)(p.s.ed + hi * kC + b * 16 + 4 * g);
            const float gm = p.s.gam[hi * DP];
            x.g[0] = f32x4{gm, gm, gm, gm};
        } else {
#pragma unroll
            for (int b = 0; b < 4; ++b) x.v[b] = *(const f32x4*)(ut + b * 16 + 4 * g);
#pragma unroll
            for (int t = 0; t < NT; ++t)
                x.g[t] = *(const f32x4*)(p.s.gam + hi * DP + min(wave + 4 * t, n_tiles - 1) * 16 + 4 * g);
        }
        const float* kt = p.s.kt + gi * DP * kC;
#pragma unroll
        for (int t = 0; t < NT; ++t) {
            const int row = min(wave + 4 * t, n_tiles - 1) * 16 + c16;  // (tiles past the state: a copy of the last one, never stored)
#pragma unroll
            for (int b = 0; b < 4; ++b) x.k[t][b] = *(const f32x4*)(kt + row * kC + b * 16 + 4 * g);
        }
    };
    auto chunk = [&](int ch, Ops& x, Ops& next) {
        const int64_t hi = (cb + ch) * a.heads + head;
        float* st = p.s.st + hi * VP * DP + (int64_t)(n0 + c16) * DP;
        if (ch + 1 < n_chunks) load(ch + 1, next);
        // S_0: to the output kernel, and to LDS as the B operand of W S_0
#pragma unroll
        for (int t = 0; t < NT; ++t)
            if (wave + 4 * t < n_tiles) {
                const int i = (wave + 4 * t) * 16 + 4 * g;
                *(f32x4*)(st + i) = S[t];
                if constexpr (KIND == MI355_REC_DELTA) *(f32x4*)(sl + c16 * ls + i) = S[t];
            }
        if constexpr (KIND == MI355_REC_DELTA) {
            lds_barrier();
            f32x4 u = zero4(), u2 = zero4();
#pragma unroll
            for (int b = 0; b < 4 * NT; ++b)
                if (b < n_tiles) {
                    const f32x4 sv = *(const f32x4*)(sl + c16 * ls + b * 16 + 4 * g);
                    if (b & 1) u2 = mfma4(x.w[b], sv, u2);
                    else u = mfma4(x.w[b], sv, u);
                }
            u = x.u - (u + u2);
            *(f32x4*)(p.s.ut + hi * VP * kC + (int64_t)(n0 + c16) * kC + wave * 16 + 4 * g) = u;
            *(f32x4*)(ul + c16 * kP + wave * 16 + 4 * g) = u * x.d;
            lds_barrier();
#pragma unroll
            for (int b = 0; b < 4; ++b) x.v[b] = *(const f32x4*)(ul + c16 * kP + b * 16 + 4 * g);
        }
        if constexpr (KIND == MI355_REC_SSD) {
#pragma unroll
            for (int b = 0; b < 4; ++b) x.v[b] *= x.e[b];
        }
#pragma unroll
        for (int t = 0; t < NT; ++t) S[t] *= x.g[kScalar ? 0 : t];
#pragma unroll
        for (int b = 0; b < 4; ++b)
#pragma unroll
            for (int t = 0; t < NT; ++t) S[t] = mfma4(x.k[t][b], x.v[b], S[t]);
    };
    Ops xa, xb;
    load(0, xa);
    for (int ch = 0; ch < n_chunks; ch += 2) {
        chunk(ch, xa, xb);
        if (ch + 1 < n_chunks) chunk(ch + 1, xb, xa);
    }
#pragma unroll
    for (int t = 0; t < NT; ++t)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const int i = (wave + 4 * t) * 16 + 4 * g + r;
            if (col_ok && i < a.dim) state[(int64_t)i * a.vdim + n0 + c16] = S[t][r];
        }
}

// ------------------------------------------------------------------------------------ outputs
// 256 threads: wave w takes the 16-column tiles w, w + 4, ...; NV = tiles per wave (VP <= 64 NV)
template <typename T, int KIND, int NV>
__global__ __launch_bounds__(256) void chunk_out_kernel(const ChunkParams p) {
    const mi355_recurrent_args& a = p.r.a;
    __shared__ float ssq[4][kC];
    int head, chunk;
    if (!head_chunk(p, head, chunk)) return;
    const int seq = p.seq0 + blockIdx.y, t0 = chunk * kC;
    const int cnt = p.r.b.count[seq];
    if (t0 >= cnt) return;
    const int DP = p.DP, VP = p.VP;
    const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
    const int c16 = lane & 15, g = lane >> 4;
    const int kvh = has_conv(KIND) ? head / (a.heads / a.kv_heads) : head;
    const int64_t ci = chunk_base(p, seq) + chunk, hi = ci * a.heads + head;
    const float* q = p.s.q + (ci * p.GQ + kvh) * kC * DP;
    const float* st = p.s.st + hi * VP * DP;
    const float* P = p.s.P + hi * kC * kC;
    const float* ut = p.s.ut + hi * VP * kC;
    const int n_tiles = VP / 16;
    f32x4 o[4][NV];
#pragma unroll
    for (int rb = 0; rb < 4; ++rb)
#pragma unroll
        for (int v = 0; v < NV; ++v) o[rb][v] = zero4();
    for (int d = 4 * g; d < DP; d += 16) {
        f32x4 b[NV];
#pragma unroll
        for (int v = 0; v < NV; ++v) b[v] = wave + 4 * v < n_tiles ? *(const f32x4*)(st + (int64_t)((wave + 4 * v) * 16 + c16) * DP + d) : zero4();
#pragma unroll
        for (int rb = 0; rb < 4; ++rb) {
            const f32x4 qv = *(const f32x4*)(q + (rb * 16 + c16) * DP + d);
#pragma unroll
            for (int v = 0; v < NV; ++v) o[rb][v] = mfma4(qv, b[v], o[rb][v]);
        }
    }
    if constexpr (has_conv(KIND)) {
#pragma unroll
        for (int rb = 0; rb < 4; ++rb) {
            const f32x4 e = *(const f32x4*)(p.s.eg + hi * kC + rb * 16 + 4 * g);
#pragma unroll
            for (int v = 0; v < NV; ++v) o[rb][v] *= e;
        }
    }
#pragma unroll
    for (int kb = 0; kb < 4; ++kb) {
        f32x4 b[NV];
#pragma unroll
        for (int v = 0; v < NV; ++v)
            b[v] = wave + 4 * v < n_tiles ? *(const f32x4*)(ut + (int64_t)((wave + 4 * v) * 16 + c16) * kC + kb * 16 + 4 * g) : zero4();
#pragma unroll
        for (int rb = kb; rb < 4; ++rb) {
            const f32x4 pv = *(const f32x4*)(P + (rb * 16 + c16) * kC + kb * 16 + 4 * g);
#pragma unroll
            for (int v = 0; v < NV; ++v) o[rb][v] = mfma4(pv, b[v], o[rb][v]);
        }
    }
    // ---- output norm over the head's columns (ssd: none), gate
    if constexpr (KIND != MI355_REC_SSD) {
#pragma unroll
        for (int rb = 0; rb < 4; ++rb)
#pragma unroll
            for (int r = 0; r < 4; ++r) {
                float s = 0.f;
#pragma unroll
                for (int v = 0; v < NV; ++v) s += o[rb][v][r] * o[rb][v][r];
                s = group_sum(s, 16);
                if (c16 == 0) ssq[wave][rb * 16 + 4 * g + r] = s;
            }
        __syncthreads();
    }
    const T* rows = (const T*)a.proj + (int64_t)(p.r.b.row0[seq] + t0) * a.ld;
    out_t<KIND, T>* y = (out_t<KIND, T>*)a.y + (int64_t)(p.r.b.row0[seq] + t0) * a.ldy;
#pragma unroll
    for (int rb = 0; rb < 4; ++rb)
#pragma unroll
        for (int r = 0; r < 4; ++r) {
            const int t = rb * 16 + 4 * g + r;
            if (t0 + t >= cnt) continue;
            const float rinv = KIND == MI355_REC_SSD ? 1.f : 1.0f / sqrtf((ssq[0][t] + ssq[1][t] + ssq[2][t] + ssq[3][t]) / (float)a.vdim + a.eps);
#pragma unroll
            for (int v = 0; v < NV; ++v) {
                const int n = (wave + 4 * v) * 16 + c16;
                if (n >= a.vdim) continue;
                const float gate = silu_f32(to_f32<T>(rows[(int64_t)t * a.ld + a.off_g + head * a.vdim + n]));
                const float w = KIND == MI355_REC_SSD ? gate : rinv * a.head_norm[head * a.norm_ld + n] * gate;
                y[(int64_t)t * a.ldy + head * a.vdim + n] = from_f32<out_t<KIND, T>>(o[rb][v][r] * w);
            }
        }
}

inline int pad16(int n) { return (n + 15) / 16 * 16; }

// floats per packed chunk
size_t chunk_floats(int kind, int heads, int kv_heads, int dim, int vdim) {
    const size_t DP = pad16(dim), VP = pad16(vdim), H = heads, G = has_conv(kind) ? kv_heads : heads;
    size_t n = 2 * G * kC * DP + H * kC * kC + H * VP * kC + H * VP * DP + H * DP;
    if (has_conv(kind)) n += G * kC * kC + 2 * H * kC;
    if (kind == MI355_REC_DELTA) n += G * kC * kC + H * kC * DP;
    return n;
}

template <typename K>
int set_lds(K kernel, size_t bytes) {
    if (bytes > 64 * 1024) {
        const hipError_t e = hipFuncSetAttribute((const void*)kernel, hipFuncAttributeMaxDynamicSharedMemorySize, (int)bytes);
        MI355_CHECK_ARG(e == hipSuccess, (int)e, "recurrent: hipFuncSetAttribute(%zu) failed: %s", bytes, hipGetErrorString(e));
    }
    return 0;
}

template <int KIND>
int launch_scan(const ChunkParams& p, int seqs, hipStream_t s) {
    const dim3 grid((p.r.a.heads + 7) / 8 * 8 * (p.VP / 16), seqs);
    const size_t lds = ((size_t)16 * (p.DP + 4) + 16 * kP) * 4;
    if (p.DP <= 64) hipLaunchKernelGGL((scan_kernel<KIND, 1>), grid, dim3(256), lds, s, p);
    else if (p.DP <= 128) hipLaunchKernelGGL((scan_kernel<KIND, 2>), grid, dim3(256), lds, s, p);
    else hipLaunchKernelGGL((scan_kernel<KIND, 4>), grid, dim3(256), lds, s, p);
    MI355_LAUNCH_CHECK();
    return 0;
}

template <typename T, int KIND>
int launch_out(const ChunkParams& p, dim3 grid, hipStream_t s) {
    if (p.VP <= 64) hipLaunchKernelGGL((chunk_out_kernel<T, KIND, 1>), grid, dim3(256), 0, s, p);
    else if (p.VP <= 128) hipLaunchKernelGGL((chunk_out_kernel<T, KIND, 2>), grid, dim3(256), 0, s, p);
    else hipLaunchKernelGGL((chunk_out_kernel<T, KIND, 4>), grid, dim3(256), 0, s, p);
    MI355_LAUNCH_CHECK();
    return 0;
}

template <typename T>
int run_group(const ChunkParams& p, int seqs, hipStream_t s) {
    const mi355_recurrent_args& a = p.r.a;
    const int chunks = (p.r.b.max_count + kC - 1) / kC;
    const dim3 heads((a.heads + 7) / 8 * 8 * chunks, seqs);
    if (a.kind == MI355_REC_DELTA) {
        const size_t lds1 = (size_t)2 * kC * (p.DP + 4) * 4;
        if (int rc = set_lds(delta_qk_kernel<T, MI355_REC_DELTA>, lds1)) return rc;
        hipLaunchKernelGGL((delta_qk_kernel<T, MI355_REC_DELTA>), dim3(chunks, a.kv_heads, seqs), dim3(256), lds1, s, p);
        MI355_LAUNCH_CHECK();
        const size_t lds2 = ((size_t)2 * kC * kP + (size_t)kC * kX + (size_t)p.VP * kP) * 4;
        if (int rc = set_lds(delta_head_kernel<T>, lds2)) return rc;
        hipLaunchKernelGGL(delta_head_kernel<T>, heads, dim3(256), lds2, s, p);
        MI355_LAUNCH_CHECK();
        if (int rc = launch_scan<MI355_REC_DELTA>(p, seqs, s)) return rc;
        return launch_out<T, MI355_REC_DELTA>(p, heads, s);
    }
    if (a.kind == MI355_REC_SSD) {
        const size_t lds = (size_t)2 * kC * (p.DP + 4) * 4;
        if (int rc = set_lds(delta_qk_kernel<T, MI355_REC_SSD>, lds)) return rc;
        hipLaunchKernelGGL((delta_qk_kernel<T, MI355_REC_SSD>), dim3(chunks, a.kv_heads, seqs), dim3(256), lds, s, p);
        MI355_LAUNCH_CHECK();
        hipLaunchKernelGGL(ssd_head_kernel<T>, heads, dim3(256), 0, s, p);
        MI355_LAUNCH_CHECK();
        if (int rc = launch_scan<MI355_REC_SSD>(p, seqs, s)) return rc;
        return launch_out<T, MI355_REC_SSD>(p, heads, s);
    }
    const size_t lds = ((size_t)3 * kC * kP + 5 * kCh + (size_t)kC * a.rank) * 4;
    if (a.kind == MI355_REC_WKV) {
        if (int rc = set_lds(gla_prep_kernel<T, MI355_REC_WKV>, lds)) return rc;
        hipLaunchKernelGGL((gla_prep_kernel<T, MI355_REC_WKV>), heads, dim3(256), lds, s, p);
    } else {
        if (int rc = set_lds(gla_prep_kernel<T, MI355_REC_GLA>, lds)) return rc;
        hipLaunchKernelGGL((gla_prep_kernel<T, MI355_REC_GLA>), heads, dim3(256), lds, s, p);
    }
    MI355_LAUNCH_CHECK();
    if (int rc = launch_scan<MI355_REC_GLA>(p, seqs, s)) return rc;
    return launch_out<T, MI355_REC_GLA>(p, heads, s);
}

}  // namespace

bool mi355_recurrent_chunks_fit(const mi355_recurrent_args& a, const mi355_seq_batch& b) {
    if (a.dim > 256 || a.vdim > 256 || a.scratch == nullptr) return false;
    return a.scratch_bytes / (chunk_floats(a.kind, a.heads, a.kv_heads, a.dim, a.vdim) * 4) >= (uint64_t)b.rows / kC + 1;
}

int mi355_recurrent_chunks(const RecParams& r, hipStream_t s) {
    const mi355_recurrent_args& a = r.a;
    ChunkParams p;
    p.r = r;
    p.DP = pad16(a.dim);
    p.VP = pad16(a.vdim);
    p.GQ = has_conv(a.kind) ? a.kv_heads : a.heads;
    const size_t per = chunk_floats(a.kind, a.heads, a.kv_heads, a.dim, a.vdim);
    // packed chunks of n sequences: at most rows / 64 + n (chunk_base)
    const size_t cap = a.scratch_bytes / (per * 4);
    const size_t most = cap - (size_t)r.b.rows / kC;  // >= 1 (mi355_recurrent_chunks_fit)
    const size_t H = a.heads, G = p.GQ, DP = p.DP, VP = p.VP;
    float* f = a.scratch;
    auto take = [&](size_t n) {
        float* q = f;
        f += n * cap;
        return q;
    };
    const bool delta = a.kind == MI355_REC_DELTA, conv = has_conv(a.kind);
    p.s.q = take(G * kC * DP);
    p.s.kt = take(G * kC * DP);
    p.s.kk = delta ? take(G * kC * kC) : nullptr;
    p.s.qk = conv ? take(G * kC * kC) : nullptr;
    p.s.P = take(H * kC * kC);
    p.s.W = delta ? take(H * kC * DP) : nullptr;
    p.s.ut = take(H * VP * kC);
    p.s.st = take(H * VP * DP);
    p.s.gam = take(H * DP);
    p.s.eg = conv ? take(H * kC) : nullptr;
    p.s.ed = conv ? take(H * kC) : nullptr;
    for (int s0 = 0; s0 < r.b.seqs; s0 += (int)most) {
        const int n = (size_t)(r.b.seqs - s0) < most ? r.b.seqs - s0 : (int)most;
        p.seq0 = s0;
        if (int rc = a.dtype == MI355_F32 ? run_group<float>(p, n, s) : run_group<bf16_t>(p, n, s)) return rc;
    }
    return 0;
}

extern "C" size_t mi355_recurrent_scratch_bytes(int kind, int rows, int seqs, int heads, int kv_heads, int dim, int vdim) {
    if (rows < 1 || seqs < 1 || heads < 1 || kv_heads < 1 || dim < 1 || vdim < 1 || dim > 256 || vdim > 256) return 0;
    return chunk_floats(kind, heads, kv_heads, dim, vdim) * 4 * ((size_t)rows / kC + seqs);
}
