// Linear recurrences with a matrix state per head: the gated delta rule (with its short convolutions), gated linear attention, WKV time
// mixing (the state in front of a token, and the token itself with a bonus per key channel), and state-space duality (short convolutions, one
// decay and one step size per head, keys and queries shared by a group of heads).
//
//   rec_rows_kernel       one workgroup per (head, sequence) walks its rows one by one with the state in registers: decode steps
//                         (convolution, gates, state update, output norm and gate in ONE launch) and short portions
//   (longer portions: recurrent_chunks.hip)
//   conv_ring_kernel      behind a portion of several rows: its last taps - 1 inputs enter the convolution's ring
//
// Everything that enters the recurrence is f32, whatever the dtype of the projections.
#include "recurrent.h"

namespace {

// state S [dim][vdim] of one (slot, head): column 64 * slice + lane, rows part * RMAX + r in registers
template <typename T, int KIND, int RMAX>
__global__ __launch_bounds__(1024) void rec_rows_kernel(const RecParams p) {
    const mi355_recurrent_args& a = p.a;
    extern __shared__ __attribute__((aligned(16))) char smem[];
    __shared__ float red[32];
    const int tid = threadIdx.x, nt = blockDim.x, lane = tid & 63;
    const int wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int slice = wave % p.slices, part = wave / p.slices;
    const int head = blockIdx.x, seq = blockIdx.y;
    const int dim = a.dim, vdim = a.vdim, kvh = head / (a.heads / a.kv_heads);
    const int pos0 = p.b.pos[seq], cnt = p.b.count[seq], slot = p.b.slot[seq];
    const int cols = p.slices * 64;
    float* q = (float*)smem;           // [parts * RMAX], zero past dim
    float* k = q + p.parts * RMAX;
    float* al = k + p.parts * RMAX;    // GLA, WKV: per-channel decay
    float* uk = al + p.parts * RMAX;   // WKV: u k
    float* pa = uk + p.parts * RMAX;   // [parts][cols] partial S^T k (DELTA)
    float* pb = pa + p.parts * cols;   // [parts][cols] partial S^T q
    float* lr = pb + p.parts * cols;   // [kMaxRank] low-rank row (GLA, WKV)

    const T* rows = (const T*)a.proj + (int64_t)p.b.row0[seq] * a.ld;
    const int ring_ld = 2 * a.kv_heads * dim + a.heads * vdim;
    T* ring = (T*)a.conv_ring + (int64_t)slot * a.taps * ring_ld;
    float* state = a.state + ((int64_t)slot * a.heads + head) * dim * vdim;
    const int col = slice * 64 + lane;
    const bool col_ok = col < vdim;

    float S[RMAX];
#pragma unroll
    for (int r = 0; r < RMAX; ++r) {
        const int i = part * RMAX + r;
        S[r] = (col_ok && i < dim) ? state[(int64_t)i * vdim + col] : 0.f;
    }
    for (int i = tid; i < p.parts * RMAX; i += nt) q[i] = k[i] = al[i] = uk[i] = 0.f;
    __syncthreads();

    for (int t = 0; t < cnt; ++t) {
        const T* row = rows + (int64_t)t * a.ld;
        // ---- the row's q, k (and decays) into LDS
        // (what needs no LDS is requested here, in front of the barriers: one memory latency instead of one per use)
        const bool out_ok = part == 0 && col_ok;
        float gate = out_ok ? silu_f32(to_f32<T>(row[a.off_g + head * vdim + col])) : 0.f;
        if constexpr (KIND != MI355_REC_SSD) gate *= out_ok ? a.head_norm[head * a.norm_ld + col] : 0.f;
        float g = 1.f, beta = 1.f, v = 0.f;
        if constexpr (KIND == MI355_REC_DELTA) {
            const float dt = softplus_f32(to_f32<T>(row[a.off_a + head]) + a.dt_bias[head]);
            g = expf(-expf(a.a_log[head]) * dt);
            beta = sigmoid_f32(to_f32<T>(row[a.off_b + head]));
            if (col_ok) {
                const int c = head * vdim + col;
                v = conv_at<T>(a, rows, ring, ring_ld, a.off_v + c, 2 * a.kv_heads * dim + c, a.conv_v + (int64_t)c * a.taps, t, pos0);
            }
            float sq = 0.f, sk = 0.f;
            for (int d = tid; d < dim; d += nt) {
                const int c = kvh * dim + d;
                const float qv = conv_at<T>(a, rows, ring, ring_ld, a.off_q + c, c, a.conv_q + (int64_t)c * a.taps, t, pos0);
                const float kv = conv_at<T>(a, rows, ring, ring_ld, a.off_k + c, a.kv_heads * dim + c, a.conv_k + (int64_t)c * a.taps, t, pos0);
                q[d] = qv;
                k[d] = kv;
                sq += qv * qv;
                sk += kv * kv;
            }
            sq = block_sum(sq, red);
            sk = block_sum(sk, red);
            const float iq = a.q_scale / sqrtf(sq + a.unit_eps), ik = 1.0f / sqrtf(sk + a.unit_eps);
            for (int d = tid; d < dim; d += nt) {
                q[d] *= iq;
                k[d] *= ik;
            }
        } else if constexpr (KIND == MI355_REC_SSD) {
            const float dt = softplus_f32(to_f32<T>(row[a.off_a + head]) + a.dt_bias[head]);
            g = expf(-expf(a.a_log[head]) * dt);
            if (col_ok) {
                const int c = head * vdim + col;
                v = conv_at<T>(a, rows, ring, ring_ld, a.off_v + c, 2 * a.kv_heads * dim + c, a.conv_v + (int64_t)c * a.taps, t, pos0, conv_bias(a.conv_bv, c));
            }
            for (int i = tid; i < 2 * dim; i += nt) {
                const bool key = i >= dim;
                const int d = key ? i - dim : i, c = kvh * dim + d;
                const float y = conv_at<T>(a, rows, ring, ring_ld, (key ? a.off_k : a.off_q) + c, (key ? a.kv_heads * dim : 0) + c,
                                           (key ? a.conv_k : a.conv_q) + (int64_t)c * a.taps, t, pos0, conv_bias(key ? a.conv_bk : a.conv_bq, c));
                if (key) k[d] = y * dt;
                else q[d] = y;
            }
        } else {
            if (col_ok) v = to_f32<T>(row[a.off_v + head * vdim + col]);
            for (int r = tid; r < a.rank; r += nt) {
                const float lv = to_f32<T>(row[a.off_a + r]);
                lr[r] = KIND == MI355_REC_WKV ? tanhf(lv) : lv;
            }
            __syncthreads();
            for (int d = tid; d < dim; d += nt) {
                const int c = head * dim + d;
                float z = a.a2_bias[c];
#pragma unroll 8
                for (int r = 0; r < a.rank; ++r) z += a.a2[(int64_t)c * a.rank + r] * lr[r];
                al[d] = expf(KIND == MI355_REC_WKV ? wkv_log_decay(z) : -softplus_f32(-z) * a.inv_tau);
                q[d] = to_f32<T>(row[a.off_q + c]) * a.q_scale;
                const float kv = to_f32<T>(row[a.off_k + c]);
                k[d] = kv;
                if constexpr (KIND == MI355_REC_WKV) uk[d] = a.bonus[c] * kv;
            }
        }
        __syncthreads();
        // ---- state update and read-out
        const float* kp = k + part * RMAX;
        const float* qp = q + part * RMAX;
        float o = 0.f;
        if constexpr (KIND == MI355_REC_DELTA) {
            float sk = 0.f;
#pragma unroll
            for (int r = 0; r < RMAX; ++r) {
                S[r] *= g;
                sk += S[r] * kp[r];
            }
            pa[part * cols + col] = sk;
            __syncthreads();
            sk = 0.f;
            for (int j = 0; j < p.parts; ++j) sk += pa[j * cols + col];
            const float u = beta * (v - sk);
#pragma unroll
            for (int r = 0; r < RMAX; ++r) {
                S[r] += kp[r] * u;
                o += S[r] * qp[r];
            }
        } else if constexpr (KIND == MI355_REC_SSD) {
#pragma unroll
            for (int r = 0; r < RMAX; ++r) {
                S[r] = g * S[r] + kp[r] * v;
                o += S[r] * qp[r];
            }
        } else if constexpr (KIND == MI355_REC_WKV) {
            const float* ap = al + part * RMAX;
            const float* up = uk + part * RMAX;
#pragma unroll
            for (int r = 0; r < RMAX; ++r) {
                o += (S[r] + up[r] * v) * qp[r];
                S[r] = ap[r] * S[r] + kp[r] * v;
            }
        } else {
            const float* ap = al + part * RMAX;
#pragma unroll
            for (int r = 0; r < RMAX; ++r) {
                S[r] = ap[r] * S[r] + kp[r] * v;
                o += S[r] * qp[r];
            }
        }
        pb[part * cols + col] = o;
        __syncthreads();
        // ---- output norm over vdim, gate (part 0 holds the columns)
        o = 0.f;
        for (int j = 0; j < p.parts; ++j) o += pb[j * cols + col];
        if constexpr (KIND == MI355_REC_SSD) {
            if (out_ok) ((float*)a.y)[(int64_t)(p.b.row0[seq] + t) * a.ldy + head * vdim + col] = (o + a.skip[head] * v) * gate;
        } else {
            const float ss = block_sum(out_ok ? o * o : 0.f, red);
            if (out_ok) {
                const float rinv = 1.0f / sqrtf(ss / (float)vdim + a.eps);
                ((T*)a.y)[(int64_t)(p.b.row0[seq] + t) * a.ldy + head * vdim + col] = from_f32<T>(o * rinv * gate);
            }
        }
        __syncthreads();
    }
#pragma unroll
    for (int r = 0; r < RMAX; ++r) {
        const int i = part * RMAX + r;
        if (col_ok && i < dim) state[(int64_t)i * vdim + col] = S[r];
    }
    // ---- a decode step's own inputs enter the ring here (row pos0 % taps held position pos0 - taps: nobody reads it any more)
    if constexpr (has_conv(KIND)) {
        if (p.b.max_count == 1) {
            T* dst = ring + (int64_t)(pos0 % a.taps) * ring_ld;
            if (head % (a.heads / a.kv_heads) == 0)
                for (int d = tid; d < dim; d += nt) {
                    dst[kvh * dim + d] = rows[a.off_q + kvh * dim + d];
                    dst[(a.kv_heads + kvh) * dim + d] = rows[a.off_k + kvh * dim + d];
                }
            for (int d = tid; d < vdim; d += nt) dst[2 * a.kv_heads * dim + head * vdim + d] = rows[a.off_v + head * vdim + d];
        }
    }
}

// grid (taps, seqs, column parts): the last rows of every portion
template <typename T>
__global__ __launch_bounds__(256) void conv_ring_kernel(const RecParams p) {
    const mi355_recurrent_args& a = p.a;
    const int seq = blockIdx.y, i = p.b.count[seq] - 1 - (int)blockIdx.x;
    if (i < 0) return;
    const int nqk = a.kv_heads * a.dim, nv = a.heads * a.vdim, ring_ld = 2 * nqk + nv;
    const T* src = (const T*)a.proj + (int64_t)(p.b.row0[seq] + i) * a.ld;
    T* dst = (T*)a.conv_ring + ((int64_t)p.b.slot[seq] * a.taps + (p.b.pos[seq] + i) % a.taps) * ring_ld;
    for (int c = blockIdx.z * 256 + threadIdx.x; c < ring_ld; c += 256 * gridDim.z)
        dst[c] = c < nqk ? src[a.off_q + c] : c < 2 * nqk ? src[a.off_k + c - nqk] : src[a.off_v + c - 2 * nqk];
}

template <typename T, int KIND, int RMAX>
int launch_rows(const RecParams& p, hipStream_t s) {
    const size_t lds = ((size_t)4 * p.parts * RMAX + (size_t)2 * p.parts * p.slices * 64 + kMaxRank) * 4;
    hipLaunchKernelGGL((rec_rows_kernel<T, KIND, RMAX>), dim3(p.a.heads, p.b.seqs), dim3(64 * p.parts * p.slices), lds, s, p);
    MI355_LAUNCH_CHECK();
    return 0;
}

template <typename T, int KIND>
int run_rows(RecParams p, hipStream_t s) {
    p.slices = (p.a.vdim + 63) / 64;
    MI355_CHECK_ARG(p.slices <= 16, MI355_E_SHAPE, "recurrent: value size %d exceeds 1024", p.a.vdim);
    // waves: up to 16, rows per thread 64 at most
    p.parts = 16 / p.slices;
    if (p.parts > 8) p.parts = 8;
    int rmax = (p.a.dim + p.parts - 1) / p.parts;
    while (p.parts > 1 && (p.a.dim + p.parts / 2 - 1) / (p.parts / 2) <= 8) {  // short states: fewer waves
        p.parts /= 2;
        rmax = (p.a.dim + p.parts - 1) / p.parts;
    }
    MI355_CHECK_ARG(rmax <= 64, MI355_E_SHAPE, "recurrent: a state of %d x %d does not fit the row kernel's registers", p.a.dim, p.a.vdim);
    int rc;
    if (rmax <= 4) rc = launch_rows<T, KIND, 4>(p, s);
    else if (rmax <= 8) rc = launch_rows<T, KIND, 8>(p, s);
    else if (rmax <= 16) rc = launch_rows<T, KIND, 16>(p, s);
    else if (rmax <= 32) rc = launch_rows<T, KIND, 32>(p, s);
    else rc = launch_rows<T, KIND, 64>(p, s);
    return rc;
}

template <typename T>
int run(const RecParams& p, hipStream_t s) {
    const bool fit = mi355_recurrent_chunks_fit(p.a, p.b);
    MI355_CHECK_ARG(p.a.path != 2 || fit, MI355_E_SHAPE, "recurrent: chunks take states of up to 256 x 256 and their scratch");
    const bool chunks = p.a.path == 2 || (p.a.path == 0 && fit && p.b.max_count > 8);
    if (chunks) {
        if (int rc = mi355_recurrent_chunks(p, s)) return rc;
    } else if (int rc = p.a.kind == MI355_REC_DELTA ? run_rows<T, MI355_REC_DELTA>(p, s)
                        : p.a.kind == MI355_REC_WKV ? run_rows<T, MI355_REC_WKV>(p, s)
                        : p.a.kind == MI355_REC_SSD ? run_rows<T, MI355_REC_SSD>(p, s)
                                                    : run_rows<T, MI355_REC_GLA>(p, s)) {
        return rc;
    }
    if (has_conv(p.a.kind) && (chunks || p.b.max_count > 1)) {
        hipLaunchKernelGGL(conv_ring_kernel<T>, dim3(p.a.taps < p.b.max_count ? p.a.taps : p.b.max_count, p.b.seqs, 16), dim3(256), 0, s, p);
        MI355_LAUNCH_CHECK();
    }
    return 0;
}

}  // namespace

extern "C" int mi355_recurrent(const mi355_recurrent_args* a, const mi355_seq_batch* b, mi355_stream_t stream) {
    MI355_CHECK_ARG(a && b && a->proj && a->state && a->y && (a->head_norm || a->kind == MI355_REC_SSD), MI355_E_ARG, "recurrent: null argument");
    MI355_CHECK_ARG(b->row0 && b->count && b->slot && b->pos, MI355_E_ARG, "recurrent: null batch");
    MI355_CHECK_ARG(b->rows > 0 && b->seqs > 0 && b->seqs <= 65535 && b->seqs <= b->rows && b->max_count > 0, MI355_E_SHAPE,
                    "recurrent: bad batch (%d rows, %d sequences)", b->rows, b->seqs);
    MI355_CHECK_ARG(a->kind >= MI355_REC_DELTA && a->kind <= MI355_REC_SSD, MI355_E_ARG, "recurrent: bad kind %d", a->kind);
    MI355_CHECK_ARG(a->dtype == MI355_F32 || a->dtype == MI355_BF16, MI355_E_DTYPE, "recurrent: dtype must be f32 or bf16");
    MI355_CHECK_ARG(a->heads > 0 && a->kv_heads > 0 && a->heads % a->kv_heads == 0 && a->dim > 0 && a->vdim > 0, MI355_E_SHAPE,
                    "recurrent: bad heads %d / %d or sizes %d / %d", a->heads, a->kv_heads, a->dim, a->vdim);
    if (has_conv(a->kind))
        MI355_CHECK_ARG(a->taps > 0 && a->conv_q && a->conv_k && a->conv_v && a->conv_ring && a->a_log && a->dt_bias, MI355_E_ARG,
                        "recurrent: the delta rule and state-space duality need their convolutions and decays");
    else
        MI355_CHECK_ARG(a->rank > 0 && a->rank <= kMaxRank && a->a2 && a->a2_bias && a->kv_heads == a->heads, MI355_E_ARG,
                        "recurrent: gated linear attention needs its decay projection (rank 1..%d)", kMaxRank);
    MI355_CHECK_ARG(a->kind != MI355_REC_WKV || a->bonus, MI355_E_ARG, "recurrent: WKV needs its bonus");
    MI355_CHECK_ARG(a->kind != MI355_REC_SSD || a->skip, MI355_E_ARG, "recurrent: state-space duality needs its skip factors");
    RecParams p;
    p.a = *a;
    p.b = *b;
    if (!has_conv(a->kind)) p.a.taps = 1;
    p.parts = p.slices = 1;
    return a->dtype == MI355_F32 ? run<float>(p, (hipStream_t)stream) : run<bf16_t>(p, (hipStream_t)stream);
}
