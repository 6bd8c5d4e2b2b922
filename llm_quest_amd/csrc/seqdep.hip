// Row operations of hybrid decoders whose sublayers run in PARALLEL off one norm and whose stream is a weighted average over depth, served in ragged batches
// (gfx950 only):
//   * the sum of both sublayers' outputs (each with its layer scale) onto the stream, the average over every earlier layer's result, and the RMS norm of that
//     average for the next layer -- one kernel;
//   * the join of differential attention: difference of two maps, unit RMS per head, sigmoid gate.
//
// Conventions as in seqmix.hip / seqrec.hip / seqpar.hip: operands come as bf16 or fp32 (a MI355_DT_* code each); stream, results, sums and norm statistics
// are fp32 in both modes.
#include "common.h"

#define ST(s) ((hipStream_t)(s))

__device__ __forceinline__ float ldd_dt(const void* p, int dt, int64_t i) { return dt == MI355_DT_F32 ? ((const float*)p)[i] : bf2f(((const bf16_t*)p)[i]); }
__device__ __forceinline__ void std_dt(void* p, int dt, int64_t i, float v) {
    if (dt == MI355_DT_F32) ((float*)p)[i] = v;
    else ((bf16_t*)p)[i] = f2bf(v);
}
__device__ __forceinline__ f32x4 ldd4_dt(const void* p, int dt, int64_t i) {
    if (dt == MI355_DT_F32) return *(const f32x4*)((const float*)p + i);
    const u32x2 r = *(const u32x2*)((const bf16_t*)p + i);
    return f32x4{__uint_as_float(r[0] << 16), __uint_as_float(r[0] & 0xffff0000u), __uint_as_float(r[1] << 16), __uint_as_float(r[1] & 0xffff0000u)};
}
__device__ __forceinline__ void std4_dt(void* p, int dt, int64_t i, f32x4 v) {
    if (dt == MI355_DT_F32) *(f32x4*)((float*)p + i) = v;
    else *(u32x2*)((bf16_t*)p + i) = u32x2{pack_bf2(v[0], v[1]), pack_bf2(v[2], v[3])};
}
static inline bool dep_dt_ok(int dt) { return dt == MI355_DT_BF16 || dt == MI355_DT_F32; }
static inline bool dep_al16(const void* p) { return ((uintptr_t)p & 15) == 0; }
static inline int dep_grid(int64_t items, int per_block, int cap) {
    int64_t g = (items + per_block - 1) / per_block;
    return (int)(g < 1 ? 1 : (g > cap ? cap : g));
}

// ------------------------------------------------------------------------------------------- parallel-sublayer sum, depth average, norm
// v = x[t] + ls1 * (ca ya[t] + cb yb[t]) + ls2 * sum_{p < parts} y2[t * parts + p];  hist[n][t] <- v;
// xa = sum_{j < n} d[j] hist[j][t] + d[n] v (no d: xa = v);  x_out <- xa;  out / out32 <- xa / sqrt(mean(xa^2) + eps) * w.
struct DepthArgs {
    const float* x;
    const void *ya, *yb, *y2;
    int64_t ldya, ldyb, ldy2, hist_stride;
    int ya_dt, yb_dt, y2_dt, parts, n_hist, out_dt;
    const float *ls1, *ls2, *d, *w;
    float* hist;
    float* x_out;
    void* out;
    float* out32;
    float ca, cb, eps;
};

// 16-byte accesses; WPR waves share a row (1: four rows per workgroup; 4: one), a lane owns NIT x 4 entries, which stay in registers from the sum to the norm.
template <int WPR, int NIT>
__global__ __launch_bounds__(256) void depth_sum_vec_kernel(int64_t T, int width, DepthArgs p) {
    __shared__ float red[4];
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    constexpr int ROWS = 4 / WPR;
    const int64_t t_step = (int64_t)gridDim.x * ROWS;
    const int i0 = WPR == 1 ? lane * 4 : threadIdx.x * 4;
    const int64_t t_first = (int64_t)blockIdx.x * ROWS + (WPR == 1 ? wave : 0);
    for (int64_t t = t_first; t < T; t += t_step) {  // WPR == 4: block-uniform, all four waves take the same trips
        f32x4 xa[NIT];
        float s = 0.f;
#pragma unroll
        for (int it = 0; it < NIT; ++it) {
            const int i = i0 + it * WPR * 256;
            f32x4 v = {0.f, 0.f, 0.f, 0.f};
            if (i < width) {
                v = *(const f32x4*)(p.x + t * width + i);
                if (p.ya) {
                    f32x4 y = p.ca * ldd4_dt(p.ya, p.ya_dt, t * p.ldya + i);
                    if (p.yb) y += p.cb * ldd4_dt(p.yb, p.yb_dt, t * p.ldyb + i);
                    v += p.ls1 ? *(const f32x4*)(p.ls1 + i) * y : y;
                }
                if (p.y2) {
                    f32x4 y = {0.f, 0.f, 0.f, 0.f};
                    for (int q = 0; q < p.parts; ++q) y += ldd4_dt(p.y2, p.y2_dt, (t * p.parts + q) * p.ldy2 + i);
                    v += p.ls2 ? *(const f32x4*)(p.ls2 + i) * y : y;
                }
                if (p.d) {
                    float* hp = p.hist + t * width + i;
                    *(f32x4*)(hp + p.n_hist * p.hist_stride) = v;
                    f32x4 a = {0.f, 0.f, 0.f, 0.f};
                    for (int j = 0; j < p.n_hist; ++j) a += p.d[j] * *(const f32x4*)(hp + j * p.hist_stride);
                    v = a + p.d[p.n_hist] * v;
                }
                if (p.x_out) *(f32x4*)(p.x_out + t * width + i) = v;
            }
            xa[it] = v;
            s += (v[0] * v[0] + v[1] * v[1]) + (v[2] * v[2] + v[3] * v[3]);
        }
        if (!p.w) continue;
        s = wave_sum(s);
        if constexpr (WPR == 4) {
            if (lane == 0) red[wave] = s;
            __syncthreads();
            s = (red[0] + red[1]) + (red[2] + red[3]);
            __syncthreads();  // red[] is reused by the next row
        }
        const float r = 1.0f / sqrtf(s / (float)width + p.eps);
#pragma unroll
        for (int it = 0; it < NIT; ++it) {
            const int i = i0 + it * WPR * 256;
            if (i >= width) continue;
            const f32x4 h = xa[it] * r * *(const f32x4*)(p.w + i);
            if (p.out) std4_dt(p.out, p.out_dt, t * width + i, h);
            if (p.out32) *(f32x4*)(p.out32 + t * width + i) = h;
        }
    }
}

// Any width and alignment: one workgroup per row, the averaged row kept in LDS.
__global__ __launch_bounds__(256) void depth_sum_kernel(int64_t T, int width, DepthArgs p) {
    extern __shared__ float row[];
    __shared__ float red[4];
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    for (int64_t t = blockIdx.x; t < T; t += gridDim.x) {
        float s = 0.f;
        for (int i = threadIdx.x; i < width; i += 256) {
            float v = p.x[t * width + i];
            if (p.ya) {
                float y = p.ca * ldd_dt(p.ya, p.ya_dt, t * p.ldya + i);
                if (p.yb) y += p.cb * ldd_dt(p.yb, p.yb_dt, t * p.ldyb + i);
                v += p.ls1 ? p.ls1[i] * y : y;
            }
            if (p.y2) {
                float y = 0.f;
                for (int q = 0; q < p.parts; ++q) y += ldd_dt(p.y2, p.y2_dt, (t * p.parts + q) * p.ldy2 + i);
                v += p.ls2 ? p.ls2[i] * y : y;
            }
            if (p.d) {
                float* hp = p.hist + t * width + i;
                hp[p.n_hist * p.hist_stride] = v;
                float a = 0.f;
                for (int j = 0; j < p.n_hist; ++j) a += p.d[j] * hp[j * p.hist_stride];
                v = a + p.d[p.n_hist] * v;
            }
            if (p.x_out) p.x_out[t * width + i] = v;
            row[i] = v;
            s += v * v;
        }
        if (!p.w) continue;
        s = wave_sum(s);
        if (lane == 0) red[wave] = s;
        __syncthreads();
        const float r = 1.0f / sqrtf(((red[0] + red[1]) + (red[2] + red[3])) / (float)width + p.eps);
        for (int i = threadIdx.x; i < width; i += 256) {  // a thread reads the entries it wrote itself
            const float h = row[i] * r * p.w[i];
            if (p.out) std_dt(p.out, p.out_dt, t * width + i, h);
            if (p.out32) p.out32[t * width + i] = h;
        }
        __syncthreads();  // red[] is reused by the next row
    }
}

extern "C" int mi355_depth_sum(int64_t tokens, int width, const float* x, const void* ya, int ya_dt, int64_t ldya, float ca, const void* yb, int yb_dt, int64_t ldyb, float cb,
                               const float* ls1, const void* y2, int y2_dt, int64_t ldy2, int parts, const float* ls2, float* hist, int64_t hist_stride, int n_hist,
                               const float* d, float* x_out, const float* w, float eps, void* out, int out_dt, float* out32, void* stream) {
    MI355_REQUIRE(tokens > 0 && width > 0 && width <= 16384 && x, "depth_sum: bad arguments (width <= 16384)");
    MI355_REQUIRE((!ya || (dep_dt_ok(ya_dt) && ldya >= width)) && (!yb || (ya && dep_dt_ok(yb_dt) && ldyb >= width)) && (!y2 || (dep_dt_ok(y2_dt) && ldy2 >= width && parts >= 1)),
                  "depth_sum: bad summands (a second branch comes with a first one)");
    MI355_REQUIRE(!d || (hist && n_hist >= 0 && hist_stride >= tokens * width), "depth_sum: a depth average needs the earlier results");
    MI355_REQUIRE((!w || out || out32) && (!out || (w && dep_dt_ok(out_dt))) && (!out32 || w), "depth_sum: the norm takes a weight and an output");
    DepthArgs p;
    p.x = x, p.ya = ya, p.yb = yb, p.y2 = y2, p.ldya = ldya, p.ldyb = ldyb, p.ldy2 = ldy2, p.hist_stride = hist_stride;
    p.ya_dt = ya_dt, p.yb_dt = yb_dt, p.y2_dt = y2_dt, p.parts = parts, p.n_hist = n_hist, p.out_dt = out_dt;
    p.ls1 = ls1, p.ls2 = ls2, p.d = d, p.w = w, p.hist = hist, p.x_out = x_out, p.out = out, p.out32 = out32, p.ca = ca, p.cb = cb, p.eps = eps;
    const bool vec = width % 4 == 0 && width <= 8192 && dep_al16(x) && dep_al16(x_out) && dep_al16(ya) && dep_al16(yb) && dep_al16(y2) && dep_al16(hist) && hist_stride % 4 == 0 &&
                     dep_al16(ls1) && dep_al16(ls2) && dep_al16(w) && dep_al16(out) && dep_al16(out32) && ldya % 4 == 0 && ldyb % 4 == 0 && ldy2 % 4 == 0;
    const int g4 = dep_grid(tokens, 4, 65535 * 8), g1 = dep_grid(tokens, 1, 65535 * 8);
    hipStream_t st = ST(stream);
    if (!vec) depth_sum_kernel<<<g1, 256, sizeof(float) * width, st>>>(tokens, width, p);
    else if (width <= 256) depth_sum_vec_kernel<1, 1><<<g4, 256, 0, st>>>(tokens, width, p);
    else if (width <= 512) depth_sum_vec_kernel<1, 2><<<g4, 256, 0, st>>>(tokens, width, p);
    else if (width <= 1024) depth_sum_vec_kernel<4, 1><<<g1, 256, 0, st>>>(tokens, width, p);
    else if (width <= 2048) depth_sum_vec_kernel<4, 2><<<g1, 256, 0, st>>>(tokens, width, p);
    else if (width <= 4096) depth_sum_vec_kernel<4, 4><<<g1, 256, 0, st>>>(tokens, width, p);
    else depth_sum_vec_kernel<4, 8><<<g1, 256, 0, st>>>(tokens, width, p);
    MI355_LAUNCH_CHECK("depth_sum");
    return 0;
}

// ------------------------------------------------------------------------------------------- join of differential attention
// Per head of D entries: o = a1 - lam * a2, o / sqrt(mean(o^2) + eps) * c, times sigmoid(gate) element by element.
struct DiffArgs {
    const float *a1, *a2;
    int64_t lda1, lda2, ldg, ldo;
    const void* gate;
    void* out;
    int H, D, g_dt, out_dt;
    float lam, eps, c;
};
// LPH lanes (a power of two) per head, four entries each, NIT trips; 64 / LPH heads per wave.
template <int NIT>
__global__ __launch_bounds__(256) void diff_join_vec_kernel(int64_t items, int LPH, DiffArgs p) {
    const int lane = threadIdx.x & 63, sub = lane & (LPH - 1);
    const int hpw = 64 / LPH;
    for (int64_t it0 = ((int64_t)blockIdx.x * 4 + (threadIdx.x >> 6)) * hpw; it0 < items; it0 += (int64_t)gridDim.x * 4 * hpw) {  // wave-uniform
        const int64_t item = it0 + lane / LPH;
        const bool ok = item < items;
        const int64_t t = ok ? item / p.H : 0;
        const int h0 = ok ? (int)(item % p.H) * p.D : 0;
        f32x4 o[NIT];
        float s = 0.f;
#pragma unroll
        for (int q = 0; q < NIT; ++q) {
            const int i = 4 * (sub + q * LPH);
            f32x4 v = {0.f, 0.f, 0.f, 0.f};
            if (ok && i < p.D) v = *(const f32x4*)(p.a1 + t * p.lda1 + h0 + i) - p.lam * *(const f32x4*)(p.a2 + t * p.lda2 + h0 + i);
            o[q] = v;
            s += (v[0] * v[0] + v[1] * v[1]) + (v[2] * v[2] + v[3] * v[3]);
        }
        for (int of = LPH >> 1; of > 0; of >>= 1) s += __shfl_xor(s, of, 64);
        const float r = p.c / sqrtf(s / (float)p.D + p.eps);
#pragma unroll
        for (int q = 0; q < NIT; ++q) {
            const int i = 4 * (sub + q * LPH);
            if (!ok || i >= p.D) continue;
            f32x4 v = o[q] * r;
            if (p.gate) {
                const f32x4 g = ldd4_dt(p.gate, p.g_dt, t * p.ldg + h0 + i);
#pragma unroll
                for (int e = 0; e < 4; ++e) v[e] *= 1.0f / (1.0f + expf(-g[e]));
            }
            std4_dt(p.out, p.out_dt, t * p.ldo + h0 + i, v);
        }
    }
}
__global__ __launch_bounds__(256) void diff_join_kernel(int64_t items, DiffArgs p) {
    const int lane = threadIdx.x & 63;
    for (int64_t item = (int64_t)blockIdx.x * 4 + (threadIdx.x >> 6); item < items; item += (int64_t)gridDim.x * 4) {
        const int64_t t = item / p.H;
        const int h0 = (int)(item % p.H) * p.D;
        const float *a1 = p.a1 + t * p.lda1 + h0, *a2 = p.a2 + t * p.lda2 + h0;
        float s = 0.f;
        for (int i = lane; i < p.D; i += 64) {
            const float v = a1[i] - p.lam * a2[i];
            s += v * v;
        }
        const float r = p.c / sqrtf(wave_sum(s) / (float)p.D + p.eps);
        for (int i = lane; i < p.D; i += 64) {
            float v = (a1[i] - p.lam * a2[i]) * r;
            if (p.gate) v *= 1.0f / (1.0f + expf(-ldd_dt(p.gate, p.g_dt, t * p.ldg + h0 + i)));
            std_dt(p.out, p.out_dt, t * p.ldo + h0 + i, v);
        }
    }
}

extern "C" int mi355_diff_join(int64_t tokens, int H, int D, const float* a1, int64_t lda1, const float* a2, int64_t lda2, float lam, float eps, float c, const void* gate, int g_dt,
                               int64_t ldg, void* out, int out_dt, int64_t ldo, void* stream) {
    const int64_t n = (int64_t)H * D;
    MI355_REQUIRE(tokens > 0 && H > 0 && D > 0 && a1 && a2 && out && dep_dt_ok(out_dt) && (!gate || (dep_dt_ok(g_dt) && ldg >= n)) && lda1 >= n && lda2 >= n && ldo >= n,
                  "diff_join: bad arguments");
    DiffArgs p;
    p.a1 = a1, p.a2 = a2, p.lda1 = lda1, p.lda2 = lda2, p.ldg = ldg, p.ldo = ldo, p.gate = gate, p.out = out, p.H = H, p.D = D, p.g_dt = g_dt, p.out_dt = out_dt;
    p.lam = lam, p.eps = eps, p.c = c;
    const int64_t items = tokens * H;
    const bool vec = D % 4 == 0 && D <= 1024 && dep_al16(a1) && dep_al16(a2) && dep_al16(gate) && dep_al16(out) && lda1 % 4 == 0 && lda2 % 4 == 0 && ldg % 4 == 0 && ldo % 4 == 0;
    if (!vec) {
        diff_join_kernel<<<dep_grid(items, 4, 65535 * 8), 256, 0, ST(stream)>>>(items, p);
    } else {
        int lph = 1;
        while (lph < 64 && lph * 4 < D) lph *= 2;
        const int grid = dep_grid(items, 4 * (64 / lph), 65535 * 8);
        if (D <= 256) diff_join_vec_kernel<1><<<grid, 256, 0, ST(stream)>>>(items, lph, p);
        else diff_join_vec_kernel<4><<<grid, 256, 0, ST(stream)>>>(items, lph, p);
    }
    MI355_LAUNCH_CHECK("diff_join");
    return 0;
}
