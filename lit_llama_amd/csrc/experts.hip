// Mixture of experts: a router over the normalised row (sigmoids, or a softmax with corrected choices inside the best groups), the `top` chosen
// experts' feed-forwards (gated SiLU, or squared ReLU) summed by weight, experts that are the row itself, and an optional shared expert that every
// row runs; the sum joins the residual stream or is stored.
//
//   route_rows_kernel    RMSNorm, router and choice of 1 to 16 rows per workgroup (router weights bf16 on the matrix cores, f32 sums)
//   choose_rows_kernel   the choice alone, where norm and router are another launch's: a wave per row
//   few rows (decode):   up_rows_kernel, down_rows_kernel: a workgroup per (row tile, chosen expert, row) / (row tile, row), every weight
//                        piece read once per row that chose its expert; three launches in all
//   many rows:           plan_kernel sorts the (row, choice) pairs by expert and cuts them into tiles; grouped_kernel multiplies a tile of up
//                        to 128 rows of one expert per workgroup; combine_kernel adds a row's experts by weight
//   exact_* kernels      f32 models: true f32, a wave per output
//
// Weights of a bf16 model are the BF16 streams of the dense linears ([tile of 16 rows][unit of 128 columns][r][piece][lane][16 B]), the
// experts' one behind the other; gate and up are a pair stream.
#include "common.h"

namespace {

constexpr int kMaxExperts = 1024, kMaxTop = 64;
constexpr int kFewRows = 2;   // rows up to which every (row, choice) pair reads its weights by itself
constexpr int kTPW = 2;       // 16-row tile slots per wave of the grouped product

__host__ __device__ __forceinline__ int pad_to(int n, int m) { return (n + m - 1) / m * m; }
__device__ __forceinline__ bf16_t bf16_hw(float f) { return __builtin_bit_cast(bf16_t, (__bf16)f); }
__device__ __forceinline__ uint32_t pack2(float a, float b) { return (uint32_t)bf16_hw(a) | ((uint32_t)bf16_hw(b) << 16); }
__device__ __forceinline__ float silu_mul(float a, float b) {
    return (a * __builtin_amdgcn_rcpf(1.0f + __builtin_amdgcn_exp2f(a * -1.44269504088896340736f))) * b;
}

struct Tile {      // up to BM rows of one expert
    int expert, m0, rows;       // sorted rows m0 .. m0 + rows - 1
    int first, count;           // the expert's tiles
    int pad[3];
};

struct Params {
    mi355_experts_args a;
    int kp, fp, fsp, np;        // width and the experts' ff in whole units of 128, width in whole tiles of 16
    int outputs;                // of the router: experts, then those that are the row itself
    bf16_t* xn;                 // [rows][ldxn] normalised rows (f32 models: float)
    int64_t ldxn;
    int32_t* ids;               // [rows][top]
    float* weights;             // [rows][top]
    bf16_t* hid;                // [rows * top][fp] (f32 models: float [rows * top][ff])
    bf16_t* hid_s;              // [rows][fsp]
    bf16_t* out;                // [rows * top][np]
    bf16_t* out_s;              // [rows][np]
    int32_t* perm;              // [rows * top] sorted position -> row
    int32_t* place;             // [rows * top] (row, choice) -> sorted position
    int32_t* n_tiles;
    Tile* tiles;
    int64_t up_bytes, down_bytes;  // one expert's streams
};

// ------------------------------------------------------------------------------------ router
// largest value of a wave, in every lane
__device__ __forceinline__ float wave_top(float v) {
    v = MI355_DPP_MAX(v, 0xB1);
    v = MI355_DPP_MAX(v, 0x4E);
    v = MI355_DPP_MAX(v, 0x141);
    v = MI355_DPP_MAX(v, 0x140);
    v = fmaxf(v, lane_xor16(v));
    return fmaxf(v, lane_xor32(v));
}

// a wave's own LDS writes are in place before it reads them
__device__ __forceinline__ void wave_lds_sync() {
    __builtin_amdgcn_fence(__ATOMIC_RELEASE, "wavefront");
    __builtin_amdgcn_wave_barrier();
    __builtin_amdgcn_fence(__ATOMIC_ACQUIRE, "wavefront");
}

// floats of LDS that choose() takes per row next to the logits
__host__ __device__ __forceinline__ int choose_floats(const mi355_experts_args& a, int E) {
    return a.score == MI355_SCORE_SIGMOID ? 0 : E + (a.keep_groups > 0 ? a.groups : 0);
}

// One wave: a row's experts and weights from its logits z[0 .. E) (LDS, overwritten; lowest index first among equals); `more`: choose_floats
__device__ __forceinline__ void choose(const mi355_experts_args& a, float* z, float* more, int E, int32_t* ids, float* weights) {
    const int lane = threadIdx.x & 63, top = a.top;
    float* s = more;         // SOFTMAX: scores, without the correction
    if (a.score == MI355_SCORE_SOFTMAX) {
        float m = -INFINITY;
        for (int e = lane; e < E; e += 64) m = fmaxf(m, z[e]);
        m = wave_top(m);
        float total = 0.f;
        for (int e = lane; e < E; e += 64) {
            const float v = expf(z[e] - m);
            s[e] = v;
            total += v;
        }
        total = group_sum(total, 64);
        for (int e = lane; e < E; e += 64) {
            const float v = s[e] / total;
            s[e] = v;
            z[e] = a.correction != nullptr ? v + a.correction[e] : v;
        }
        if (a.keep_groups > 0) {
            float* best = more + E;  // per group
            const int size = E / a.groups;
            wave_lds_sync();
            for (int g = lane; g < a.groups; g += 64) {
                float v = -INFINITY;
                for (int e = g * size; e < (g + 1) * size; ++e) v = fmaxf(v, z[e]);
                best[g] = v;
            }
            wave_lds_sync();
            for (int e = lane; e < E; e += 64) {
                const int g = e / size;
                const float mine = best[g];
                int ahead = 0;
                for (int o = 0; o < a.groups; ++o) ahead += best[o] > mine || (best[o] == mine && o < g);
                if (ahead >= a.keep_groups) z[e] = -INFINITY;
            }
        }
        wave_lds_sync();
    }
    float best = -INFINITY;
    int bi = lane < E ? lane : E - 1;  // (rows of NaNs)
    auto scan = [&] {
        best = -INFINITY;
        for (int e = lane; e < E; e += 64) {
            const float v = z[e];
            if (v > best) best = v, bi = e;
        }
    };
    scan();
    float mine = -INFINITY;
    int my_id = 0;
    for (int k = 0; k < top; ++k) {
        const float v = wave_top(best);
        unsigned long long at = __ballot(best == v);
        if (at == 0) at = 1;
        int i = __builtin_amdgcn_readlane(bi, __builtin_ctzll(at));
        for (unsigned long long more_at = at & (at - 1); more_at != 0; more_at &= more_at - 1) i = min(i, __builtin_amdgcn_readlane(bi, __builtin_ctzll(more_at)));
        if (lane == k) mine = v, my_id = i;
        if (lane == (i & 63)) {
            z[i] = -INFINITY;
            scan();
        }
    }
    if (a.score == MI355_SCORE_SOFTMAX) {
        if (lane < top) {
            ids[lane] = my_id;
            weights[lane] = s[my_id] * a.scale;
        }
        return;
    }
    const float sg = lane < top ? 1.0f / (1.0f + expf(-mine)) : 0.f;
    const float total = group_sum(sg, 64);
    if (lane < top) {
        ids[lane] = my_id;
        weights[lane] = sg / (total + 1e-20f) * a.scale;
    }
}

// grid ceil(rows / 4), 256 threads.  LDS: per wave the logits and choose_floats
__global__ __launch_bounds__(256) void choose_rows_kernel(const Params p) {
    const mi355_experts_args& a = p.a;
    extern __shared__ __attribute__((aligned(16))) char smem[];
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, row = blockIdx.x * 4 + wave, E = p.outputs;
    if (row >= a.rows) return;
    float* z = (float*)smem + wave * (E + choose_floats(a, E));
    const float* from = a.logits + (int64_t)row * a.ld_logits;
    for (int e = lane; e < E; e += 64) z[e] = from[e];
    wave_lds_sync();
    choose(a, z, z + E, E, p.ids + (int64_t)row * a.top, p.weights + (int64_t)row * a.top);
}

// grid ceil(rows / R), 512 threads; R = 1, 2, 4, 8, 16.  LDS: partial logits [8 waves][tiles of a pass][256], logits [R][outputs + 1], choose_floats [R]
constexpr int kRouteTiles = 2;
template <int R>
__global__ __launch_bounds__(512) void route_rows_kernel(const Params p) {
    const mi355_experts_args& a = p.a;
    constexpr int kPer = R < 8 ? 8 / R : 1, kRows = R > 8 ? R / 8 : 1;  // waves per row, rows per wave
    extern __shared__ __attribute__((aligned(16))) char smem[];
    __shared__ float sums[8];
    const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6);
    const int g = lane >> 4, c = lane & 15;
    const int row0 = blockIdx.x * R;
    const int W = a.width, E = p.outputs, tiles = (E + 15) / 16, pass = tiles < kRouteTiles ? tiles : kRouteTiles;
    float* part = (float*)smem;
    float* z = part + 8 * pass * 256;
    // a wave's first router weights are requested ahead of the norm, the next unit's ahead of a unit's products (past the last tile or unit:
    // the last one again, not used)
    const int units = p.kp / 128;
    const uint8_t* wr = (const uint8_t*)a.router + lane * 16;
    auto wload = [&](int t, int u, int d) {
        return *(const bf16x8*)(wr + ((int64_t)(min(t, tiles - 1) * units + min(u, units - 1)) * 4 + d) * 1024);
    };
    bf16x8 wn[kRouteTiles][4];
#pragma unroll
    for (int t = 0; t < kRouteTiles; ++t)
#pragma unroll
        for (int d = 0; d < 4; ++d) wn[t][d] = wload(t, wave, d);

#pragma unroll
    for (int i = 0; i < kRows; ++i) {
        const int row = row0 + wave / kPer + 8 * i, share = wave % kPer;
        const bool live = row < a.rows;
        const float* x = a.x + (int64_t)(live ? row : row0) * a.ldx;
        bf16_t* o = p.xn + (int64_t)row * p.ldxn;
        const bool vec = W % 4 == 0 && a.norm_dtype == MI355_BF16;
        constexpr int kHeld = 16 / kPer, kStep = 64 * kPer;  // (rows of 4096; what lies behind is read twice)
        f32x4 v[kHeld];
        u32x2 n[kHeld];
        float ss = 0.f;
        if (vec) {
#pragma unroll
            for (int h = 0; h < kHeld; ++h) {
                const int j = min(share * 64 + lane + h * kStep, W / 4 - 1);
                v[h] = ((const f32x4*)x)[j];
                n[h] = ((const u32x2*)a.norm)[j];
            }
#pragma unroll
            for (int h = 0; h < kHeld; ++h) {
                const float q = (v[h][0] * v[h][0] + v[h][1] * v[h][1]) + (v[h][2] * v[h][2] + v[h][3] * v[h][3]);
                ss += share * 64 + lane + h * kStep < W / 4 ? q : 0.f;
            }
            for (int j = share * 64 + lane + kHeld * kStep; j < W / 4; j += kStep) {
                const f32x4 t = ((const f32x4*)x)[j];
                ss += (t[0] * t[0] + t[1] * t[1]) + (t[2] * t[2] + t[3] * t[3]);
            }
        } else {
            for (int k = share * 64 + lane; k < W; k += kStep) ss += x[k] * x[k];
        }
        ss = group_sum(ss, 64);
        if constexpr (kPer > 1) {
            if (lane == 0) sums[wave] = ss;
            __syncthreads();
            ss = 0.f;
#pragma unroll
            for (int s = 0; s < kPer; ++s) ss += sums[wave / kPer * kPer + s];
        }
        const float rinv = 1.0f / sqrtf(ss / (float)W + a.eps);
        if (live && vec) {
            auto put = [&](int j, f32x4 t, u32x2 m) {
                u32x2 q = {pack2(t[0] * rinv * (a.norm_add + __uint_as_float(m[0] << 16)), t[1] * rinv * (a.norm_add + __uint_as_float(m[0] & 0xffff0000u))),
                           pack2(t[2] * rinv * (a.norm_add + __uint_as_float(m[1] << 16)), t[3] * rinv * (a.norm_add + __uint_as_float(m[1] & 0xffff0000u)))};
                if (j >= W / 4) q = u32x2{0u, 0u};
                if (j < p.kp / 4) ((u32x2*)o)[j] = q;
            };
#pragma unroll
            for (int h = 0; h < kHeld; ++h) put(share * 64 + lane + h * kStep, v[h], n[h]);
            for (int j = share * 64 + lane + kHeld * kStep; j < p.kp / 4; j += kStep) {
                const int i4 = min(j, W / 4 - 1);
                put(j, ((const f32x4*)x)[i4], ((const u32x2*)a.norm)[i4]);
            }
        } else if (live) {
            for (int k = share * 64 + lane; k < p.kp; k += kStep)
                o[k] = k < W ? bf16_hw(x[k] * rinv * (a.norm_add + ld_as_f32(a.norm, k, a.norm_dtype))) : (bf16_t)0;
        }
    }
    __syncthreads();
    const int row = min(row0 + c % R, a.rows - 1);
    const bf16_t* xr = p.xn + (int64_t)row * p.ldxn + 32 * g;
    for (int t0 = 0; t0 < tiles; t0 += pass) {
        f32x4 acc[kRouteTiles];
#pragma unroll
        for (int t = 0; t < kRouteTiles; ++t) acc[t] = f32x4{0.f, 0.f, 0.f, 0.f};
        for (int u = wave; u < units; u += 8) {
            bf16x8 b[4], w[kRouteTiles][4];
#pragma unroll
            for (int d = 0; d < 4; ++d) b[d] = *(const bf16x8*)(xr + u * 128 + 8 * d);
#pragma unroll
            for (int t = 0; t < kRouteTiles; ++t)
#pragma unroll
                for (int d = 0; d < 4; ++d) w[t][d] = wn[t][d];
            const bool more = u + 8 < units;  // (else the next pass begins)
#pragma unroll
            for (int t = 0; t < kRouteTiles; ++t)
#pragma unroll
                for (int d = 0; d < 4; ++d) wn[t][d] = wload(more ? t0 + t : t0 + pass + t, more ? u + 8 : wave, d);
#pragma unroll
            for (int d = 0; d < 4; ++d)
#pragma unroll
                for (int t = 0; t < kRouteTiles; ++t) acc[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(w[t][d], b[d], acc[t], 0, 0, 0);
        }
#pragma unroll
        for (int t = 0; t < kRouteTiles; ++t)
            if (t < pass) *(f32x4*)(part + (wave * pass + t) * 256 + lane * 4) = acc[t];
        __syncthreads();
        for (int i = threadIdx.x; i < pass * 256; i += 512) {
            const int l = (i & 255) >> 2, e = (t0 + (i >> 8)) * 16 + 4 * (l >> 4) + (i & 3);
            if ((l & 15) >= R || e >= E) continue;
            float s = 0.f;
#pragma unroll
            for (int w = 0; w < 8; ++w) s += part[w * pass * 256 + i];
            z[(l & 15) * (E + 1) + e] = s;
        }
        __syncthreads();
    }
    for (int r = wave; r < R && row0 + r < a.rows; r += 8)
        choose(a, z + r * (E + 1), z + R * (E + 1) + r * choose_floats(a, E), E, p.ids + (int64_t)(row0 + r) * a.top, p.weights + (int64_t)(row0 + r) * a.top);
}

// f32 models: one row per workgroup.  LDS: the normalised row, the logits, choose_floats
__global__ __launch_bounds__(256) void exact_route_kernel(const Params p) {
    const mi355_experts_args& a = p.a;
    extern __shared__ __attribute__((aligned(16))) char smem[];
    __shared__ float red[32];
    float *h = (float*)smem, *z = h + a.width;
    const int row = blockIdx.x, lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    const float* x = a.x + (int64_t)row * a.ldx;
    float ss = 0.f;
    for (int k = threadIdx.x; k < a.width; k += 256) ss += x[k] * x[k];
    const float rinv = 1.0f / sqrtf(block_sum(ss, red) / (float)a.width + a.eps);
    float* o = (float*)p.xn + (int64_t)row * p.ldxn;
    for (int k = threadIdx.x; k < a.width; k += 256) o[k] = h[k] = x[k] * rinv * (a.norm_add + ld_as_f32(a.norm, k, a.norm_dtype));
    __syncthreads();
    for (int e = wave; e < p.outputs; e += 4) {
        const float* w = (const float*)a.router + (int64_t)e * a.width;
        float s = 0.f;
        for (int k = lane; k < a.width; k += 64) s += w[k] * h[k];
        s = group_sum(s, 64);
        if (lane == 0) z[e] = s;
    }
    __syncthreads();
    if (wave == 0) choose(a, z, z + p.outputs, p.outputs, p.ids + (int64_t)row * a.top, p.weights + (int64_t)row * a.top);
}

// column n of a row's sum
__device__ __forceinline__ void put_sum(const mi355_experts_args& a, int row, int n, float v) {
    if (a.out != nullptr) a.out[(int64_t)row * a.ld_out + n] = a.alpha * v;
    else a.x[(int64_t)row * a.ldx + n] += a.alpha * v;
}

// ------------------------------------------------------------------------------------ f32 experts: a wave per output
// grid (ceil(widest ff / 4), choices (+ 1), rows)
__global__ __launch_bounds__(256) void exact_up_kernel(const Params p) {
    const mi355_experts_args& a = p.a;
    const int lane = threadIdx.x & 63, n = blockIdx.x * 4 + (threadIdx.x >> 6), k = blockIdx.y, row = blockIdx.z;
    const bool shared = k == a.top;
    const int ff = shared ? a.ff_shared : a.ff;
    if (n >= ff) return;
    const int64_t slot = (int64_t)row * a.top + k;
    if (!shared && p.ids[slot] >= a.experts) return;  // (the row itself)
    const float* w = shared ? (const float*)a.shared_up : (const float*)a.up + (int64_t)p.ids[slot] * (a.act == MI355_ACT_RELU2 ? 1 : 2) * a.ff * a.width;
    if (a.act == MI355_ACT_RELU2) {
        const float *wu = w + (int64_t)n * a.width, *h = (const float*)p.xn + (int64_t)row * p.ldxn;
        float s = 0.f;
        for (int j = lane; j < a.width; j += 64) s += wu[j] * h[j];
        s = group_sum(s, 64);
        if (lane == 0) ((float*)p.hid + slot * ff)[n] = relu2_f32(s);
        return;
    }
    const float *wg = w + (int64_t)n * a.width, *wu = wg + (int64_t)ff * a.width, *h = (const float*)p.xn + (int64_t)row * p.ldxn;
    float sg = 0.f, su = 0.f;
    for (int j = lane; j < a.width; j += 64) sg += wg[j] * h[j], su += wu[j] * h[j];
    sg = group_sum(sg, 64), su = group_sum(su, 64);
    if (lane == 0) (shared ? (float*)p.hid_s + (int64_t)row * ff : (float*)p.hid + slot * ff)[n] = swiglu_f32(sg, su);
}

// grid (ceil(width / 4), rows)
__global__ __launch_bounds__(256) void exact_down_kernel(const Params p) {
    const mi355_experts_args& a = p.a;
    const int lane = threadIdx.x & 63, n = blockIdx.x * 4 + (threadIdx.x >> 6), row = blockIdx.y;
    if (n >= a.width) return;
    float total = 0.f;
    for (int k = 0; k < a.top + (a.ff_shared > 0); ++k) {
        const bool shared = k == a.top;
        const int ff = shared ? a.ff_shared : a.ff;
        const int64_t slot = (int64_t)row * a.top + k;
        if (!shared && p.ids[slot] >= a.experts) {
            total += p.weights[slot] * ((const float*)p.xn)[(int64_t)row * p.ldxn + n];
            continue;
        }
        const float* w = (shared ? (const float*)a.shared_down : (const float*)a.down + (int64_t)p.ids[slot] * a.width * a.ff) + (int64_t)n * ff;
        const float* h = shared ? (const float*)p.hid_s + (int64_t)row * ff : (const float*)p.hid + slot * ff;
        float s = 0.f;
        for (int j = lane; j < ff; j += 64) s += w[j] * h[j];
        total += (shared ? 1.f : p.weights[slot]) * group_sum(s, 64);
    }
    if (lane == 0) put_sum(a, row, n, total);
}

// ------------------------------------------------------------------------------------ few rows
// grid (widest fp / 16, choices (+ 1), rows), 512 threads: 16 hidden columns of one choice; the waves share the units of K.  Every column of
// the matrix instruction carries the same row.  R: matrices of the stream (2: gate and up, 1: squared ReLU)
template <int R>
__global__ __launch_bounds__(512) void up_rows_kernel(const Params p) {
    const mi355_experts_args& a = p.a;
    __shared__ float part[8][R][16];
    const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), g = lane >> 4, c = lane & 15;
    const int tile = blockIdx.x, k = blockIdx.y, row = blockIdx.z;
    const bool shared = k == a.top;
    const int fp = shared ? p.fsp : p.fp, ff = shared ? a.ff_shared : a.ff, units = p.kp / 128;
    if (tile * 16 >= fp) return;
    const int64_t slot = (int64_t)row * a.top + k;
    const int id = shared ? 0 : p.ids[slot];
    if (id >= a.experts) return;  // (the row itself)
    const uint8_t* w = shared ? (const uint8_t*)a.shared_up : (const uint8_t*)a.up + id * p.up_bytes;
    w += (int64_t)tile * units * R * 4096 + lane * 16;
    const bf16_t* x = p.xn + (int64_t)row * p.ldxn + 32 * g;
    f32x4 acc[R];
#pragma unroll
    for (int r = 0; r < R; ++r) acc[r] = f32x4{0.f, 0.f, 0.f, 0.f};
    if (tile * 16 < ff) {
#pragma unroll 2
        for (int u = wave; u < units; u += 8) {
            u32x4 q[R][4];
            bf16x8 b[4];
#pragma unroll
            for (int r = 0; r < R; ++r)
#pragma unroll
                for (int d = 0; d < 4; ++d) q[r][d] = *(const u32x4*)(w + (int64_t)u * R * 4096 + r * 4096 + d * 1024);
#pragma unroll
            for (int d = 0; d < 4; ++d) b[d] = *(const bf16x8*)(x + u * 128 + 8 * d);
#pragma unroll
            for (int d = 0; d < 4; ++d)
#pragma unroll
                for (int r = 0; r < R; ++r)
                    acc[r] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(bf16x8, q[r][d]), b[d], acc[r], 0, 0, 0);
        }
    }
    if (c == 0) {
#pragma unroll
        for (int r = 0; r < R; ++r)
#pragma unroll
            for (int i = 0; i < 4; ++i) part[wave][r][4 * g + i] = acc[r][i];
    }
    __syncthreads();
    if (threadIdx.x < 16) {
        float s[R];
#pragma unroll
        for (int r = 0; r < R; ++r) {
            s[r] = 0.f;
#pragma unroll
            for (int w8 = 0; w8 < 8; ++w8) s[r] += part[w8][r][threadIdx.x];
        }
        (shared ? p.hid_s + (int64_t)row * fp : p.hid + slot * fp)[tile * 16 + threadIdx.x] = bf16_hw(R == 2 ? silu_mul(s[0], s[R - 1]) : relu2_f32(s[0]));
    }
}

// grid (np / 16, rows), 512 threads: 16 columns of one row; the waves share the (choice, unit) pairs
__global__ __launch_bounds__(512) void down_rows_kernel(const Params p) {
    const mi355_experts_args& a = p.a;
    __shared__ float part[8][16];
    const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), g = lane >> 4, c = lane & 15;
    const int tile = blockIdx.x, row = blockIdx.y;
    __shared__ int real[kMaxTop], n_real;
    const int64_t slot0 = (int64_t)row * a.top;
    if (a.identity > 0) {  // the choices that have weights
        if (threadIdx.x < 64) {
            const bool has = lane < a.top && p.ids[slot0 + min(lane, a.top - 1)] < a.experts;
            const unsigned long long all = __ballot(has);
            if (has) real[__popcll(all & ((1ull << lane) - 1))] = lane;
            if (lane == 0) n_real = __popcll(all);
        }
        __syncthreads();
    }
    const int units = p.fp / 128, units_s = p.fsp / 128, routed = (a.identity > 0 ? n_real : a.top) * units, items = routed + units_s;
    f32x4 total = {0.f, 0.f, 0.f, 0.f};
#pragma unroll 2
    for (int i = wave; i < items; i += 8) {
        const bool shared = i >= routed;
        const int at = shared ? a.top : i / units, u = shared ? i - routed : i - at * units;
        const int k = a.identity > 0 && !shared ? real[at] : at;
        const uint8_t* w = shared ? (const uint8_t*)a.shared_down + ((int64_t)tile * units_s + u) * 4096
                                  : (const uint8_t*)a.down + p.ids[slot0 + k] * p.down_bytes + ((int64_t)tile * units + u) * 4096;
        const bf16_t* h = (shared ? p.hid_s + (int64_t)row * p.fsp : p.hid + (slot0 + k) * p.fp) + u * 128 + 32 * g;
        const float f = shared ? 1.f : p.weights[slot0 + k];
        f32x4 acc = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int d = 0; d < 4; ++d)
            acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(*(const bf16x8*)(w + d * 1024 + lane * 16), *(const bf16x8*)(h + 8 * d), acc, 0, 0, 0);
#pragma unroll
        for (int r = 0; r < 4; ++r) total[r] += f * acc[r];
    }
    if (c == 0) {
#pragma unroll
        for (int i = 0; i < 4; ++i) part[wave][4 * g + i] = total[i];
    }
    __syncthreads();
    const int n = tile * 16 + threadIdx.x;
    if (threadIdx.x < 16 && n < a.width) {
        float s = 0.f;
#pragma unroll
        for (int w8 = 0; w8 < 8; ++w8) s += part[w8][threadIdx.x];
        for (int k = 0; a.identity > 0 && k < a.top; ++k)
            if (p.ids[slot0 + k] >= a.experts) s += p.weights[slot0 + k] * bf16_to_f32(p.xn[(int64_t)row * p.ldxn + n]);
        put_sum(a, row, n, s);
    }
}

// ------------------------------------------------------------------------------------ many rows
// one workgroup: (row, choice) pairs sorted by expert, tiles of up to bm rows of one expert
__global__ __launch_bounds__(1024) void plan_kernel(const Params p, int bm) {
    const mi355_experts_args& a = p.a;
    __shared__ int count[kMaxExperts], rows_to[kMaxExperts], tiles_to[kMaxExperts];
    const int tid = threadIdx.x, pairs = a.rows * a.top;
    count[tid] = 0;
    __syncthreads();
    for (int i = tid; i < pairs; i += 1024)  // (experts that are the row itself have nothing to multiply)
        if (p.ids[i] < a.experts) atomicAdd(&count[p.ids[i]], 1);
    __syncthreads();
    const int n = count[tid], t = (n + bm - 1) / bm;
    rows_to[tid] = n;
    tiles_to[tid] = t;
    __syncthreads();
    for (int o = 1; o < kMaxExperts; o <<= 1) {  // inclusive sums
        const int r = tid >= o ? rows_to[tid - o] : 0, q = tid >= o ? tiles_to[tid - o] : 0;
        __syncthreads();
        rows_to[tid] += r;
        tiles_to[tid] += q;
        __syncthreads();
    }
    const int m0 = rows_to[tid] - n, t0 = tiles_to[tid] - t;
    for (int j = 0; j < t; ++j) {
        Tile x = {tid, m0 + j * bm, n - j * bm < bm ? n - j * bm : bm, t0, t, {0, 0, 0}};
        p.tiles[t0 + j] = x;
    }
    if (tid == kMaxExperts - 1) *p.n_tiles = tiles_to[tid];
    count[tid] = m0;
    __syncthreads();
    for (int i = tid; i < pairs; i += 1024) {
        if (p.ids[i] >= a.experts) {
            p.place[i] = -1;
            continue;
        }
        const int at = atomicAdd(&count[p.ids[i]], 1);
        p.perm[at] = i / a.top;
        p.place[i] = at;
    }
}

// the same 16-byte chunk swizzle of an activation row in LDS as the dense product's (gemm.hip)
__device__ __forceinline__ int swz(int tok) { return (tok & 3) ^ (((tok >> 2) & 1) << 3) ^ (((tok >> 3) & 1) * 12); }

struct Grouped {
    const uint8_t *w, *w_s;     // first expert's stream, the shared expert's
    int64_t group_bytes;        // one expert's stream
    unsigned bytes_s;
    int real, real_s;           // row tiles of the streams
    int tiles, tiles_s;         // row tiles written (UP: whole units of hidden columns, zeros behind the stream's)
    int units, units_s;
    const bf16_t *x, *x_s;
    int64_t ldx, ldx_s;
    unsigned xbytes, xbytes_s;
    bf16_t *y, *y_s;
    int64_t ldy, ldy_s;
};

// UP: rows gathered by p.perm, the activation stored (kUpPair: pair stream, SiLU(gate) up; kUpOne: squared ReLU); kDown: rows as sorted, plain sums
// stored.  A workgroup: BM rows x kWaves pairs of row tiles (kUpPair: one tile of both matrices).  Operands of the next unit: rows by LDS-DMA, weights into the registers the unit before left
enum { kDown = 0, kUpPair = 1, kUpOne = 2 };
template <int UP, int BM, int kWaves>
__global__ __launch_bounds__(64 * kWaves) void grouped_kernel(const Params p, const Grouped q) {
    constexpr bool kPair = UP == kUpPair;
    constexpr int kTT = BM / 16, kThreads = 64 * kWaves, kChunks = BM * 16 / kThreads, kPer = kPair ? kWaves : kWaves * kTPW;
    extern __shared__ __attribute__((aligned(16))) char smem[];
    const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), g = lane >> 4, c = lane & 15;
    const int n_e = *p.n_tiles, n_s = p.a.ff_shared > 0 ? (p.a.rows + BM - 1) / BM : 0;
    const int nb_e = (q.tiles + kPer - 1) / kPer, nb_s = (q.tiles_s + kPer - 1) / kPer;
    const int total = n_e * nb_e + n_s * nb_s, per_xcd = (total + 7) / 8;
    // workgroup b runs on XCD b % 8, which takes a contiguous range of (expert, row block, token tile)
    const int j = blockIdx.x >> 3, L = (blockIdx.x & 7) * per_xcd + j;
    if (j >= per_xcd || L >= total) return;
    const bool shared = L >= n_e * nb_e;
    int m0, rows, nb, expert = 0;
    if (shared) {
        const int l = L - n_e * nb_e;
        nb = l / n_s;
        m0 = (l - nb * n_s) * BM;
        rows = min(BM, p.a.rows - m0);
    } else {
        const Tile any = p.tiles[L / nb_e];
        const int l = L - any.first * nb_e;
        nb = l / any.count;
        const Tile t = p.tiles[any.first + (l - nb * any.count)];
        m0 = t.m0, rows = t.rows, expert = t.expert;
    }
    const int units = shared ? q.units_s : q.units, real = shared ? q.real_s : q.real, tiles = shared ? q.tiles_s : q.tiles;
    const unsigned w_bytes = shared ? q.bytes_s : (unsigned)q.group_bytes;
    const void* w = shared ? q.w_s : q.w + expert * q.group_bytes;
    const __amdgpu_buffer_rsrc_t rw = __builtin_amdgcn_make_buffer_rsrc((void*)w, 0, (int)w_bytes, 0x00020000);
    const __amdgpu_buffer_rsrc_t none = __builtin_amdgcn_make_buffer_rsrc((void*)w, 0, 0, 0x00020000);
    const __amdgpu_buffer_rsrc_t rx =
        __builtin_amdgcn_make_buffer_rsrc((void*)(shared ? q.x_s : q.x), 0, (int)(shared ? q.xbytes_s : q.xbytes), 0x00020000);
    const int64_t ldx = shared ? q.ldx_s : q.ldx;
    int tile[kTPW];
#pragma unroll
    for (int t = 0; t < kTPW; ++t) tile[t] = kPair ? nb * kWaves + wave : nb * kPer + kTPW * wave + t;
    auto wload = [&](int t, int u, int d, u32x4& dst) {
        const bool ok = tile[t] < real && u < units;
        const unsigned off = (unsigned)((tile[t] * units + u) * (kPair ? 2 : 1) + (kPair ? t : 0)) * 4096u + d * 1024u;
        dst = __builtin_bit_cast(u32x4, __builtin_amdgcn_raw_buffer_load_b128(ok ? rw : none, lane * 16, ok ? off : 0u, 0));
    };
    unsigned xoff[kChunks];
#pragma unroll
    for (int i = 0; i < kChunks; ++i) {
        const int ch = i * kThreads + threadIdx.x, tok = ch >> 4, slot = ch & 15;
        xoff[i] = 0xFFFFFFF0u;
        if (tok < rows) {
            const int row = UP != kDown && !shared ? p.perm[m0 + tok] : m0 + tok;
            xoff[i] = (unsigned)((int64_t)row * ldx * 2) + (unsigned)((slot ^ swz(tok)) * 16);
        }
    }
    auto xdma = [&](int u, int buf) {
        if (u >= units) return;
#pragma unroll
        for (int i = 0; i < kChunks; ++i) {
            const unsigned off = xoff[i] == 0xFFFFFFF0u ? xoff[i] : xoff[i] + (unsigned)u * 256u;
            __builtin_amdgcn_raw_ptr_buffer_load_lds(rx, (__attribute__((address_space(3))) void*)(smem + buf * (BM * 256) + (i * kThreads + wave * 64) * 16),
                                                     16, off, 0, 0, 0);
        }
    };
    f32x4 acc[kTPW][kTT];
#pragma unroll
    for (int t = 0; t < kTPW; ++t)
#pragma unroll
        for (int tt = 0; tt < kTT; ++tt) acc[t][tt] = f32x4{0.f, 0.f, 0.f, 0.f};
    u32x4 wcur[kTPW][4];
#pragma unroll
    for (int t = 0; t < kTPW; ++t)
#pragma unroll
        for (int d = 0; d < 4; ++d) wload(t, 0, d, wcur[t][d]);
    xdma(0, 0);
    __syncthreads();
    for (int u = 0; u < units; ++u) {
        xdma(u + 1, (u & 1) ^ 1);
        __builtin_amdgcn_sched_barrier(0);
        const char* xs = smem + (u & 1) * (BM * 256);
#pragma unroll
        for (int d = 0; d < 4; ++d) {
            bf16x8 w8[kTPW];
#pragma unroll
            for (int t = 0; t < kTPW; ++t) w8[t] = __builtin_bit_cast(bf16x8, wcur[t][d]);
#pragma unroll
            for (int tt = 0; tt < kTT; ++tt) {
                const int tok = tt * 16 + c;
                const bf16x8 b = *(const bf16x8*)(xs + tok * 256 + (((4 * g + d) ^ swz(tok)) << 4));
#pragma unroll
                for (int t = 0; t < kTPW; ++t) acc[t][tt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(w8[t], b, acc[t][tt], 0, 0, 0);
            }
#pragma unroll
            for (int t = 0; t < kTPW; ++t) wload(t, u + 1, d, wcur[t][d]);
        }
        __syncthreads();
    }
    bf16_t* y = shared ? q.y_s : q.y;
    const int64_t ldy = shared ? q.ldy_s : q.ldy;
#pragma unroll
    for (int tt = 0; tt < kTT; ++tt) {
        const int tok = tt * 16 + c;
        if (tok >= rows) continue;
        bf16_t* dst = y + (int64_t)(m0 + tok) * ldy + 4 * g;
        if constexpr (UP == kUpOne) {
#pragma unroll
            for (int t = 0; t < kTPW; ++t)
                if (tile[t] < tiles)
                    *(u32x2*)(dst + tile[t] * 16) = u32x2{pack2(relu2_f32(acc[t][tt][0]), relu2_f32(acc[t][tt][1])),
                                                          pack2(relu2_f32(acc[t][tt][2]), relu2_f32(acc[t][tt][3]))};
        } else if constexpr (kPair) {
            if (tile[0] < tiles)
                *(u32x2*)(dst + tile[0] * 16) = u32x2{pack2(silu_mul(acc[0][tt][0], acc[1][tt][0]), silu_mul(acc[0][tt][1], acc[1][tt][1])),
                                                      pack2(silu_mul(acc[0][tt][2], acc[1][tt][2]), silu_mul(acc[0][tt][3], acc[1][tt][3]))};
        } else {
#pragma unroll
            for (int t = 0; t < kTPW; ++t)
                if (tile[t] < tiles) *(u32x2*)(dst + tile[t] * 16) = u32x2{pack2(acc[t][tt][0], acc[t][tt][1]), pack2(acc[t][tt][2], acc[t][tt][3])};
        }
    }
}

// grid rows: alpha (sum of the chosen experts' rows by weight + the shared expert's)
__global__ __launch_bounds__(256) void combine_kernel(const Params p) {
    const mi355_experts_args& a = p.a;
    __shared__ float wgt[kMaxTop];
    __shared__ int at[kMaxTop];
    const int row = blockIdx.x;
    if ((int)threadIdx.x < a.top) {
        wgt[threadIdx.x] = p.weights[(int64_t)row * a.top + threadIdx.x];
        at[threadIdx.x] = p.place[(int64_t)row * a.top + threadIdx.x];
    }
    __syncthreads();
    float* x = a.x + (int64_t)row * a.ldx;
    for (int j = threadIdx.x; j < p.np / 8; j += 256) {
        float s[8];
#pragma unroll
        for (int e = 0; e < 8; ++e) s[e] = 0.f;
        auto add = [&](const bf16_t* src, float f) {
            const u32x4 r = ((const u32x4*)src)[j];
#pragma unroll
            for (int e = 0; e < 4; ++e) s[2 * e] += f * __uint_as_float(r[e] << 16), s[2 * e + 1] += f * __uint_as_float(r[e] & 0xffff0000u);
        };
#pragma unroll 4
        for (int k = 0; k < a.top; ++k) add(at[k] >= 0 ? p.out + (int64_t)at[k] * p.np : p.xn + (int64_t)row * p.ldxn, wgt[k]);
        if (a.ff_shared > 0) add(p.out_s + (int64_t)row * p.np, 1.f);
        f32x4* o = (f32x4*)((a.out != nullptr ? a.out + (int64_t)row * a.ld_out : x) + 8 * j);  // (columns width .. np are zeros plus zeros)
#pragma unroll
        for (int h = 0; h < 2; ++h) {
            f32x4 v = a.out != nullptr ? f32x4{0.f, 0.f, 0.f, 0.f} : o[h];
#pragma unroll
            for (int e = 0; e < 4; ++e) v[e] += a.alpha * s[4 * h + e];
            o[h] = v;
        }
    }
}

// ------------------------------------------------------------------------------------ host
// lays the scratch out; returns its bytes
size_t lay_out(Params& p, char* base) {
    const mi355_experts_args& a = p.a;
    const bool exact = a.dtype == MI355_F32;
    p.kp = pad_to(a.width, 128), p.fp = pad_to(a.ff, 128), p.fsp = pad_to(a.ff_shared, 128), p.np = pad_to(a.width, 16);
    size_t at = 0;
    auto take = [&](size_t bytes) {
        char* r = base + at;
        at += (bytes + 255) & ~(size_t)255;
        return r;
    };
    const size_t rows = a.rows, pairs = rows * a.top;
    p.outputs = a.experts + a.identity;
    p.ldxn = a.h != nullptr ? a.ldh : exact ? a.width : p.kp;
    p.xn = a.h != nullptr ? (bf16_t*)a.h : (bf16_t*)take(exact ? rows * a.width * 4 : rows * p.kp * 2);
    p.hid = (bf16_t*)take(exact ? pairs * a.ff * 4 : pairs * p.fp * 2);
    p.hid_s = (bf16_t*)take(exact ? rows * a.ff_shared * 4 : rows * p.fsp * 2);
    p.ids = (int32_t*)take(pairs * 4);
    p.weights = (float*)take(pairs * 4);
    if (!exact) {
        p.out = (bf16_t*)take(pairs * p.np * 2);
        p.out_s = (bf16_t*)take(a.ff_shared > 0 ? rows * p.np * 2 : 0);
        p.perm = (int32_t*)take(pairs * 4);
        p.place = (int32_t*)take(pairs * 4);
        p.n_tiles = (int32_t*)take(4);
        p.tiles = (Tile*)take((pairs / 16 + a.experts + 1) * sizeof(Tile));
    }
    return at;
}

template <int UP, int BM, int kWaves>
int launch_grouped(const Params& p, const Grouped& q, hipStream_t s) {
    constexpr int kPer = UP == kUpPair ? kWaves : kWaves * kTPW, kLds = 2 * BM * 256;
    static hipError_t e = hipFuncSetAttribute((const void*)grouped_kernel<UP, BM, kWaves>, hipFuncAttributeMaxDynamicSharedMemorySize, kLds);
    MI355_CHECK_ARG(e == hipSuccess, (int)e, "experts: hipFuncSetAttribute failed: %s", hipGetErrorString(e));
    const int64_t pairs = (int64_t)p.a.rows * p.a.top;
    // (every expert that has rows ends with at most one tile that is not full)
    const int64_t most_e = pairs / BM + (pairs < p.a.experts ? pairs : p.a.experts), n_s = p.a.ff_shared > 0 ? (p.a.rows + BM - 1) / BM : 0;
    const int64_t grid = (most_e * ((q.tiles + kPer - 1) / kPer) + n_s * ((q.tiles_s + kPer - 1) / kPer) + 7) / 8 * 8;
    MI355_CHECK_ARG(grid < 0x7fffffff, MI355_E_SHAPE, "experts: grid of %lld workgroups", (long long)grid);
    hipLaunchKernelGGL((grouped_kernel<UP, BM, kWaves>), dim3((unsigned)grid), dim3(64 * kWaves), kLds, s, p, q);
    MI355_LAUNCH_CHECK();
    return 0;
}

template <int UP>
int run_grouped(const Params& p, const Grouped& q, int bm, hipStream_t s) {
    if (bm == 128) return launch_grouped<UP, 128, 8>(p, q, s);
    if (bm == 64) return launch_grouped<UP, 64, 8>(p, q, s);
    return launch_grouped<UP, 16, 4>(p, q, s);
}

int run_many(Params& p, hipStream_t s) {
    const mi355_experts_args& a = p.a;
    const int64_t pairs = (int64_t)a.rows * a.top;
    const int bm = pairs >= (int64_t)96 * a.experts ? 128 : pairs >= (int64_t)32 * a.experts ? 64 : 16;
    hipLaunchKernelGGL(plan_kernel, dim3(1), dim3(1024), 0, s, p, bm);
    MI355_LAUNCH_CHECK();
    Grouped q;
    memset(&q, 0, sizeof(q));
    q.w = (const uint8_t*)a.up, q.w_s = (const uint8_t*)a.shared_up, q.group_bytes = p.up_bytes;
    q.units = q.units_s = p.kp / 128;
    q.real = (a.ff + 15) / 16, q.real_s = (a.ff_shared + 15) / 16, q.tiles = p.fp / 16, q.tiles_s = p.fsp / 16;
    q.bytes_s = (unsigned)((size_t)q.real_s * q.units * 8192);
    q.x = q.x_s = p.xn, q.ldx = q.ldx_s = p.ldxn, q.xbytes = q.xbytes_s = (unsigned)((size_t)a.rows * p.ldxn * 2);
    q.y = p.hid, q.ldy = p.fp, q.y_s = p.hid_s, q.ldy_s = p.fsp;
    if (int rc = a.act == MI355_ACT_RELU2 ? run_grouped<kUpOne>(p, q, bm, s) : run_grouped<kUpPair>(p, q, bm, s)) return rc;
    q.w = (const uint8_t*)a.down, q.w_s = (const uint8_t*)a.shared_down, q.group_bytes = p.down_bytes;
    q.units = p.fp / 128, q.units_s = p.fsp / 128;
    q.real = q.tiles = p.np / 16;
    q.real_s = q.tiles_s = a.ff_shared > 0 ? p.np / 16 : 0;
    q.bytes_s = (unsigned)((size_t)q.real_s * q.units_s * 4096);
    q.x = p.hid, q.ldx = p.fp, q.xbytes = (unsigned)((size_t)pairs * p.fp * 2);
    q.x_s = p.hid_s, q.ldx_s = p.fsp, q.xbytes_s = (unsigned)((size_t)a.rows * p.fsp * 2);
    q.y = p.out, q.y_s = p.out_s, q.ldy = q.ldy_s = p.np;
    if (int rc = run_grouped<kDown>(p, q, bm, s)) return rc;
    hipLaunchKernelGGL(combine_kernel, dim3(a.rows), dim3(256), 0, s, p);
    MI355_LAUNCH_CHECK();
    return 0;
}

template <int R>
int launch_route(const Params& p, hipStream_t s) {
    const mi355_experts_args& a = p.a;
    const int tiles = (p.outputs + 15) / 16, pass = tiles < kRouteTiles ? tiles : kRouteTiles;
    const size_t lds = ((size_t)8 * pass * 256 + R * (p.outputs + 1 + choose_floats(a, p.outputs))) * 4;
    MI355_CHECK_ARG(lds <= 144 * 1024, MI355_E_SHAPE, "experts: the choice of %d rows does not fit LDS", R);
    static hipError_t e = hipFuncSetAttribute((const void*)route_rows_kernel<R>, hipFuncAttributeMaxDynamicSharedMemorySize, 144 * 1024);
    MI355_CHECK_ARG(e == hipSuccess, (int)e, "experts: hipFuncSetAttribute failed: %s", hipGetErrorString(e));
    hipLaunchKernelGGL(route_rows_kernel<R>, dim3((a.rows + R - 1) / R), dim3(512), lds, s, p);
    MI355_LAUNCH_CHECK();
    return 0;
}

int run_choose(const Params& p, hipStream_t s) {
    const size_t lds = (size_t)4 * (p.outputs + choose_floats(p.a, p.outputs)) * 4;  // (at most 48 KB)
    hipLaunchKernelGGL(choose_rows_kernel, dim3((p.a.rows + 3) / 4), dim3(256), lds, s, p);
    MI355_LAUNCH_CHECK();
    return 0;
}

// rows per workgroup: as few as give every CU one workgroup
int run_route(const Params& p, hipStream_t s) {
    const int rows = p.a.rows;
    if (p.a.logits != nullptr) return run_choose(p, s);
    if (rows <= 256) return launch_route<1>(p, s);
    if (rows <= 512) return launch_route<2>(p, s);
    if (rows <= 1024) return launch_route<4>(p, s);
    if (rows <= 2048) return launch_route<8>(p, s);
    return launch_route<16>(p, s);
}

int run_few(const Params& p, hipStream_t s) {
    const mi355_experts_args& a = p.a;
    const int shared = a.ff_shared > 0, widest = p.fp > p.fsp ? p.fp : p.fsp;
    if (a.act == MI355_ACT_RELU2) hipLaunchKernelGGL(up_rows_kernel<1>, dim3(widest / 16, a.top + shared, a.rows), dim3(512), 0, s, p);
    else hipLaunchKernelGGL(up_rows_kernel<2>, dim3(widest / 16, a.top + shared, a.rows), dim3(512), 0, s, p);
    MI355_LAUNCH_CHECK();
    hipLaunchKernelGGL(down_rows_kernel, dim3(p.np / 16, a.rows), dim3(512), 0, s, p);
    MI355_LAUNCH_CHECK();
    return 0;
}

int run_exact(const Params& p, hipStream_t s) {
    const mi355_experts_args& a = p.a;
    const int shared = a.ff_shared > 0, widest = a.ff > a.ff_shared ? a.ff : a.ff_shared;
    if (a.logits != nullptr) {
        if (int rc = run_choose(p, s)) return rc;
    } else {
        const size_t lds = ((size_t)a.width + p.outputs + choose_floats(a, p.outputs)) * 4;
        MI355_CHECK_ARG(lds <= 150 * 1024, MI355_E_SHAPE, "experts: rows of %d do not fit LDS", a.width);
        static hipError_t e = hipFuncSetAttribute((const void*)exact_route_kernel, hipFuncAttributeMaxDynamicSharedMemorySize, 150 * 1024);
        MI355_CHECK_ARG(e == hipSuccess, (int)e, "experts: hipFuncSetAttribute failed: %s", hipGetErrorString(e));
        hipLaunchKernelGGL(exact_route_kernel, dim3(a.rows), dim3(256), lds, s, p);
        MI355_LAUNCH_CHECK();
    }
    hipLaunchKernelGGL(exact_up_kernel, dim3((widest + 3) / 4, a.top + shared, a.rows), dim3(256), 0, s, p);
    MI355_LAUNCH_CHECK();
    hipLaunchKernelGGL(exact_down_kernel, dim3((a.width + 3) / 4, a.rows), dim3(256), 0, s, p);
    MI355_LAUNCH_CHECK();
    return 0;
}

}  // namespace

extern "C" size_t mi355_experts_scratch_bytes(const mi355_experts_args* a) {
    if (a == nullptr || a->rows <= 0 || a->width <= 0 || a->ff <= 0 || a->top <= 0) return 0;
    Params p;
    memset(&p, 0, sizeof(p));
    p.a = *a;
    return lay_out(p, nullptr);
}

extern "C" int mi355_experts(const mi355_experts_args* a, mi355_stream_t stream) {
    MI355_CHECK_ARG(a && a->up && a->down && a->scratch && (a->x || a->out), MI355_E_ARG, "experts: null argument");
    MI355_CHECK_ARG(a->logits ? a->h != nullptr : a->router != nullptr, MI355_E_ARG, "experts: logits come with the rows they were made of, or from a router");
    MI355_CHECK_ARG(a->h ? a->logits != nullptr : a->x != nullptr && a->norm != nullptr, MI355_E_ARG, "experts: rows come with their logits, or are normalised here");
    MI355_CHECK_ARG(a->dtype == MI355_F32 || a->dtype == MI355_BF16, MI355_E_DTYPE, "experts: dtype must be f32 or bf16");
    MI355_CHECK_ARG(a->rows > 0 && a->rows <= 65535 && a->width > 0 && a->ff > 0 && a->ff_shared >= 0, MI355_E_SHAPE, "experts: bad shape (%d rows of %d, ff %d / %d)",
                    a->rows, a->width, a->ff, a->ff_shared);
    MI355_CHECK_ARG(a->x == nullptr || (a->ldx >= pad_to(a->width, 16) && a->ldx % 4 == 0), MI355_E_SHAPE, "experts: bad pitch of x");
    MI355_CHECK_ARG(a->out == nullptr || (a->ld_out >= pad_to(a->width, 16) && a->ld_out % 4 == 0 && (uintptr_t)a->out % 16 == 0), MI355_E_SHAPE, "experts: bad rows of the sum");
    MI355_CHECK_ARG(a->h == nullptr || (a->dtype == MI355_F32 ? a->ldh >= a->width : a->ldh >= pad_to(a->width, 128) && a->ldh % 8 == 0 && (uintptr_t)a->h % 16 == 0),
                    MI355_E_SHAPE, "experts: bad normalised rows");
    MI355_CHECK_ARG(a->ff_shared == 0 || (a->shared_up && a->shared_down && a->act == MI355_ACT_SILU_GATE), MI355_E_ARG, "experts: bad shared expert");
    MI355_CHECK_ARG(a->experts > 0 && a->identity >= 0 && a->experts <= kMaxExperts && a->identity <= kMaxExperts - a->experts && a->top > 0 &&
                        a->top <= a->experts + a->identity && a->top <= kMaxTop,
                    MI355_E_SHAPE, "experts: %d of %d + %d (at most %d of %d)", a->top, a->experts, a->identity, kMaxTop, kMaxExperts);
    MI355_CHECK_ARG((a->score == MI355_SCORE_SIGMOID && a->correction == nullptr && a->keep_groups == 0) || a->score == MI355_SCORE_SOFTMAX, MI355_E_ARG,
                    "experts: corrections and groups belong to softmax scores");
    MI355_CHECK_ARG(a->act == MI355_ACT_SILU_GATE || a->act == MI355_ACT_RELU2, MI355_E_ARG, "experts: bad activation %d", a->act);
    MI355_CHECK_ARG(a->keep_groups == 0 || (a->keep_groups > 0 && a->groups >= a->keep_groups && (a->experts + a->identity) % a->groups == 0 &&
                                            (int64_t)a->keep_groups * ((a->experts + a->identity) / a->groups) >= a->top),
                    MI355_E_SHAPE, "experts: %d of %d groups of %d outputs", a->keep_groups, a->groups, a->experts + a->identity);
    MI355_CHECK_ARG((uintptr_t)a->x % 16 == 0 && (uintptr_t)a->norm % 8 == 0 && (uintptr_t)a->scratch % 256 == 0, MI355_E_ARG, "experts: unaligned operand");
    Params p;
    memset(&p, 0, sizeof(p));
    p.a = *a;
    const size_t need = lay_out(p, (char*)a->scratch);
    MI355_CHECK_ARG(a->scratch_bytes >= need, MI355_E_SHAPE, "experts: scratch of %llu bytes, %zu needed", (unsigned long long)a->scratch_bytes, need);
    hipStream_t s = (hipStream_t)stream;
    if (a->dtype == MI355_F32) return run_exact(p, s);
    p.up_bytes = (int64_t)((a->ff + 15) / 16) * (p.kp / 128) * (a->act == MI355_ACT_RELU2 ? 4096 : 8192);
    p.down_bytes = (int64_t)(p.np / 16) * (p.fp / 128) * 4096;
    const int64_t pairs = (int64_t)a->rows * a->top;
    MI355_CHECK_ARG(p.up_bytes < 0xFFFFFFF0ll && p.down_bytes < 0xFFFFFFF0ll && pairs * p.fp * 2 < 0xFFFFFFF0ll && (int64_t)a->rows * p.fsp * 2 < 0xFFFFFFF0ll &&
                        (int64_t)a->rows * p.ldxn * 2 < 0xFFFFFFF0ll && (int64_t)((a->ff_shared + 15) / 16) * p.kp * 64 < 0xFFFFFFF0ll &&
                        (int64_t)p.np * p.fsp * 2 < 0xFFFFFFF0ll,
                    MI355_E_SHAPE, "experts: an operand exceeds 4 GiB");
    if (int rc = run_route(p, s)) return rc;
    return a->path == 1 || (a->path == 0 && a->rows <= kFewRows) ? run_few(p, s) : run_many(p, s);
}
