// Row operations of decoders with several residual streams (hyper-connections) served in ragged batches (gfx950 only): what lies between two sublayers -- the pending
// sublayer output joins every stream, the streams mix, the next sublayer's input is read off them and normed -- is one kernel.
//
// Conventions as in seqmix.hip / seqdep.hip: operands come as bf16 or fp32 (a MI355_DT_* code each); streams, mixing and norm statistics are fp32 in both modes.
#include "common.h"

#define ST(s) ((hipStream_t)(s))

__device__ __forceinline__ float ldh_dt(const void* p, int dt, int64_t i) { return dt == MI355_DT_F32 ? ((const float*)p)[i] : bf2f(((const bf16_t*)p)[i]); }
__device__ __forceinline__ void sth_dt(void* p, int dt, int64_t i, float v) {
    if (dt == MI355_DT_F32) ((float*)p)[i] = v;
    else ((bf16_t*)p)[i] = f2bf(v);
}
__device__ __forceinline__ f32x4 ldh4_dt(const void* p, int dt, int64_t i) {
    if (dt == MI355_DT_F32) return *(const f32x4*)((const float*)p + i);
    const u32x2 r = *(const u32x2*)((const bf16_t*)p + i);
    return f32x4{__uint_as_float(r[0] << 16), __uint_as_float(r[0] & 0xffff0000u), __uint_as_float(r[1] << 16), __uint_as_float(r[1] & 0xffff0000u)};
}
__device__ __forceinline__ void sth4_dt(void* p, int dt, int64_t i, f32x4 v) {
    if (dt == MI355_DT_F32) *(f32x4*)((float*)p + i) = v;
    else *(u32x2*)((bf16_t*)p + i) = u32x2{pack_bf2(v[0], v[1]), pack_bf2(v[2], v[3])};
}
static inline bool hyp_dt_ok(int dt) { return dt == MI355_DT_BF16 || dt == MI355_DT_F32; }
static inline bool hyp_al16(const void* p) { return ((uintptr_t)p & 15) == 0; }
static inline int hyp_grid(int64_t items, int per_block, int cap) {
    int64_t g = (items + per_block - 1) / per_block;
    return (int)(g < 1 ? 1 : (g > cap ? cap : g));
}

// ------------------------------------------------------------------------------------------- streams: join, mix, read, norm
// Token t's stream s is x + t * x_ts + s * x_ss.  With a sublayer output: yv = y_scale * sum_{p < parts} y[t * parts + p], stream to <- sum_from mix[from, to] x_from +
// put[to] * yv (all from the old streams); x_out [T, S, width] receives them.  u = sum_s read[s] x_s of the streams as they now are; u_out <- u;
// out <- u / sqrt(mean(u^2) + eps) * w.  rows (optional): output row t works on token rows[t] instead of t.
struct HyperArgs {
    const float* x;
    int64_t x_ts, x_ss, ldy;
    const void* y;
    const float *mix, *put, *read, *w;
    const int64_t* rows;
    float *x_out, *u_out;
    void* out;
    int y_dt, parts, out_dt, S;
    float y_scale, eps;
};

// 16-byte accesses; WPR waves share a row (1: four rows per workgroup; 4: one), a lane owns NIT x 4 entries of every stream; u stays in registers from the sum to
// the norm.  NS streams (EXACT), or up to NS.
template <int NS, bool EXACT, int WPR, int NIT>
__global__ __launch_bounds__(256) void hyper_mix_vec_kernel(int64_t T, int width, HyperArgs p) {
    __shared__ float red[4];
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    constexpr int ROWS = 4 / WPR;
    const int S = EXACT ? NS : p.S;
    const int i0 = WPR == 1 ? lane * 4 : threadIdx.x * 4;
    const int64_t t_first = (int64_t)blockIdx.x * ROWS + (WPR == 1 ? wave : 0);
    for (int64_t t = t_first; t < T; t += (int64_t)gridDim.x * ROWS) {  // WPR == 4: block-uniform, all four waves take the same trips
        const int64_t r = p.rows ? p.rows[t] : t;
        f32x4 u[NIT];
        float ss = 0.f;
#pragma unroll
        for (int it = 0; it < NIT; ++it) {
            const int i = i0 + it * WPR * 256;
            f32x4 a = {0.f, 0.f, 0.f, 0.f};
            if (i < width) {
                f32x4 xs[NS];
#pragma unroll
                for (int s = 0; s < NS; ++s) xs[s] = EXACT || s < S ? *(const f32x4*)(p.x + r * p.x_ts + s * p.x_ss + i) : a;
                if (p.y) {
                    f32x4 yv = ldh4_dt(p.y, p.y_dt, r * p.parts * p.ldy + i);
                    for (int q = 1; q < p.parts; ++q) yv += ldh4_dt(p.y, p.y_dt, (r * p.parts + q) * p.ldy + i);
                    yv *= p.y_scale;
                    f32x4 n[NS];
#pragma unroll
                    for (int to = 0; to < NS; ++to) {
                        n[to] = a;
                        if (EXACT || to < S) {
                            f32x4 v = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
                            for (int s = 0; s < NS; ++s)
                                if (EXACT || s < S) v += p.mix[s * S + to] * xs[s];
                            n[to] = v + p.put[to] * yv;
                        }
                    }
#pragma unroll
                    for (int s = 0; s < NS; ++s) xs[s] = n[s];
                }
                if (p.x_out) {
#pragma unroll
                    for (int s = 0; s < NS; ++s)
                        if (EXACT || s < S) *(f32x4*)(p.x_out + (t * S + s) * width + i) = xs[s];
                }
                if (p.read) {
#pragma unroll
                    for (int s = 0; s < NS; ++s)
                        if (EXACT || s < S) a += p.read[s] * xs[s];
                    if (p.u_out) *(f32x4*)(p.u_out + t * width + i) = a;
                }
            }
            u[it] = a;
            ss += (a[0] * a[0] + a[1] * a[1]) + (a[2] * a[2] + a[3] * a[3]);
        }
        if (!p.w) continue;
        ss = wave_sum(ss);
        if constexpr (WPR == 4) {
            if (lane == 0) red[wave] = ss;
            __syncthreads();
            ss = (red[0] + red[1]) + (red[2] + red[3]);
            __syncthreads();  // red[] is reused by the next row
        }
        const float rn = 1.0f / sqrtf(ss / (float)width + p.eps);
#pragma unroll
        for (int it = 0; it < NIT; ++it) {
            const int i = i0 + it * WPR * 256;
            if (i < width) sth4_dt(p.out, p.out_dt, t * width + i, u[it] * rn * *(const f32x4*)(p.w + i));
        }
    }
}

// Any number of streams, any width and alignment: one workgroup per row, u kept in LDS.
__global__ __launch_bounds__(256) void hyper_mix_kernel(int64_t T, int width, HyperArgs p) {
    extern __shared__ float row[];
    __shared__ float red[4];
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    for (int64_t t = blockIdx.x; t < T; t += gridDim.x) {
        const int64_t r = p.rows ? p.rows[t] : t;
        float ss = 0.f;
        for (int i = threadIdx.x; i < width; i += 256) {
            const float* x = p.x + r * p.x_ts + i;
            float yv = 0.f, u = 0.f;
            if (p.y) {
                for (int q = 0; q < p.parts; ++q) yv += ldh_dt(p.y, p.y_dt, (r * p.parts + q) * p.ldy + i);
                yv *= p.y_scale;
            }
            for (int to = 0; to < p.S; ++to) {
                float v = 0.f;
                if (p.y) {
                    for (int s = 0; s < p.S; ++s) v += p.mix[s * p.S + to] * x[s * p.x_ss];
                    v += p.put[to] * yv;
                } else {
                    v = x[to * p.x_ss];
                }
                if (p.x_out) p.x_out[(t * p.S + to) * width + i] = v;
                if (p.read) u += p.read[to] * v;
            }
            if (p.u_out) p.u_out[t * width + i] = u;
            row[i] = u;
            ss += u * u;
        }
        if (!p.w) continue;
        ss = wave_sum(ss);
        if (lane == 0) red[wave] = ss;
        __syncthreads();
        const float rn = 1.0f / sqrtf(((red[0] + red[1]) + (red[2] + red[3])) / (float)width + p.eps);
        for (int i = threadIdx.x; i < width; i += 256) sth_dt(p.out, p.out_dt, t * width + i, row[i] * rn * p.w[i]);  // a thread reads the entries it wrote itself
        __syncthreads();  // red[] is reused by the next row
    }
}

template <int NS, bool EXACT>
static void launch_hyper(int64_t T, int width, const HyperArgs& p, hipStream_t st) {
    const int g4 = hyp_grid(T, 4, 65535 * 8), g1 = hyp_grid(T, 1, 65535 * 8);
    if (width <= 256) hyper_mix_vec_kernel<NS, EXACT, 1, 1><<<g4, 256, 0, st>>>(T, width, p);
    else if (width <= 512) hyper_mix_vec_kernel<NS, EXACT, 1, 2><<<g4, 256, 0, st>>>(T, width, p);
    else if (width <= 1024) hyper_mix_vec_kernel<NS, EXACT, 4, 1><<<g1, 256, 0, st>>>(T, width, p);
    else if (width <= 2048) hyper_mix_vec_kernel<NS, EXACT, 4, 2><<<g1, 256, 0, st>>>(T, width, p);
    else if (width <= 4096) hyper_mix_vec_kernel<NS, EXACT, 4, 4><<<g1, 256, 0, st>>>(T, width, p);
    else hyper_mix_vec_kernel<NS, EXACT, 4, 8><<<g1, 256, 0, st>>>(T, width, p);
}

extern "C" int mi355_hyper_mix(int64_t tokens, int width, int S, const float* x, int64_t x_ts, int64_t x_ss, const void* y, int y_dt, int64_t ldy, int parts, float y_scale,
                               const float* mix, const float* put, const float* read, const int64_t* rows, float* x_out, float* u_out, const float* w, float eps, void* out,
                               int out_dt, void* stream) {
    MI355_REQUIRE(tokens > 0 && width > 0 && width <= 16000 && S > 0 && S <= 1024 && x && x_ts >= 0 && x_ss >= 0, "hyper_mix: bad arguments (width <= 16000, streams <= 1024)");
    MI355_REQUIRE(!y || (hyp_dt_ok(y_dt) && ldy >= width && parts >= 1 && mix && put), "hyper_mix: a sublayer output comes with its mixing matrix and its weight per stream");
    MI355_REQUIRE((x_out || read) && x_out != x && (!u_out || read) && (!w || (read && out && hyp_dt_ok(out_dt))), "hyper_mix: streams out, or a read-out (norms and u_out take one); not in place");
    HyperArgs p;
    p.x = x, p.x_ts = x_ts, p.x_ss = x_ss, p.ldy = ldy, p.y = y, p.mix = mix, p.put = put, p.read = read, p.w = w, p.rows = rows, p.x_out = x_out, p.u_out = u_out, p.out = out;
    p.y_dt = y_dt, p.parts = parts, p.out_dt = out_dt, p.S = S, p.y_scale = y_scale, p.eps = eps;
    const bool vec = width % 4 == 0 && width <= 8192 && S <= 8 && x_ts % 4 == 0 && x_ss % 4 == 0 && ldy % 4 == 0 && hyp_al16(x) && hyp_al16(y) && hyp_al16(x_out) && hyp_al16(u_out) &&
                     hyp_al16(w) && hyp_al16(out);
    hipStream_t st = ST(stream);
    if (!vec) hyper_mix_kernel<<<hyp_grid(tokens, 1, 65535 * 8), 256, sizeof(float) * width, st>>>(tokens, width, p);
    else if (S == 1) launch_hyper<1, true>(tokens, width, p, st);
    else if (S == 2) launch_hyper<2, true>(tokens, width, p, st);
    else if (S == 3) launch_hyper<3, true>(tokens, width, p, st);
    else if (S == 4) launch_hyper<4, true>(tokens, width, p, st);
    else launch_hyper<8, false>(tokens, width, p, st);
    MI355_LAUNCH_CHECK("hyper_mix");
    return 0;
}
