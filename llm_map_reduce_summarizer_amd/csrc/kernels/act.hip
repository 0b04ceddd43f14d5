// SwiGLU activation (K7) and token-embedding gather (K9).
//
// swiglu:  gu [T, 2F] bf16, the fused gate+up GEMM output with its columns in
//          blocks of 16 = [8 gate | 8 up] (the weight layout the decode GEMM's
//          fused SwiGLU epilogue needs); out [T, F] = silu(gate) * up,
//          16-B vectors, grid-stride.
// embed:   ids [T] int32 -> out [T, D] = table[ids]; one block per token,
//          16-B vectors (a row is D*2 bytes = 8 KiB at D=4096).  Ids are
//          clamped to [0, V) so a bad id can never read out of bounds.
// embed_pos: fp32 residual rows table[id] * scale + sinusoidal position (entry 2i sin(p f_i), 2i + 1 cos(p f_i)).
//          The angle is reduced to one turn in double, so far positions lose nothing.
// embed_bigram: fp32 residual rows rms(table[id] * scale + bigram[pair of previous token and id]) * w.
// gelu_cols: columns of a projection's slabs -> tanh-form gelu into columns of the joint output rows.
// clamp_glu: [8 gate | 8 up]-blocked projection -> min(g, limit) sigmoid(alpha g) (clamp(u, -limit, limit) + shift).
#include "common.h"

// grid (F/8/256 column blocks, T rows): no 64-bit div/mod per element (a size_t i / fv here cost
// ~20 us per call at T=48, more than the memory traffic).
__global__ __launch_bounds__(256) void swiglu_kernel(const bf16* __restrict__ gu, bf16* __restrict__ out, int T,
                                                     int F) {
    const int fv = F >> 3;
    const int r = blockIdx.y;
    for (int c = blockIdx.x * 256 + threadIdx.x; c < fv; c += gridDim.x * 256) {  // output features [8c, 8c+8)
        const uint4* row = reinterpret_cast<const uint4*>(gu + r * 2 * (size_t)F);
        float g[8], u[8];  // 16-B vector 2c = gate features [8c, 8c+8), 2c+1 = the matching up
        unpack8(row[2 * c], g);
        unpack8(row[2 * c + 1], u);
#pragma unroll
        for (int j = 0; j < 8; ++j) g[j] = g[j] / (1.f + __expf(-g[j])) * u[j];
        reinterpret_cast<uint4*>(out + r * (size_t)F)[c] = pack8(g);
    }
}

MRSUM_API int mrsum_swiglu(const void* gu, void* out, int T, int F, hipStream_t s) {
    if (T <= 0) return 0;
    if (F % 8) return (int)hipErrorInvalidValue;
    const int cb = std::min(ceil_div(F / 8, 256), 64);
    for (int t0 = 0; t0 < T; t0 += 65535) {  // grid.y limit
        const int tn = std::min(T - t0, 65535);
        swiglu_kernel<<<dim3(cb, tn), 256, 0, s>>>((const bf16*)gu + (size_t)t0 * 2 * F, (bf16*)out + (size_t)t0 * F,
                                                   tn, F);
    }
    return (int)hipGetLastError();
}

__global__ __launch_bounds__(256) void embed_kernel(const int* __restrict__ ids, const bf16* __restrict__ table,
                                                    bf16* __restrict__ out, int D, int V) {
    int id = ids[blockIdx.x];
    id = id < 0 ? 0 : (id >= V ? V - 1 : id);
    const uint4* src = reinterpret_cast<const uint4*>(table + (size_t)id * D);
    uint4* dst = reinterpret_cast<uint4*>(out + (size_t)blockIdx.x * D);
    for (int c = threadIdx.x; c < (D >> 3); c += blockDim.x) dst[c] = src[c];
}

MRSUM_API int mrsum_embed(const int* ids, const void* table, void* out, int T, int D, int V, hipStream_t s) {
    if (T <= 0) return 0;
    if (D % 8) return (int)hipErrorInvalidValue;
    embed_kernel<<<T, 256, 0, s>>>(ids, (const bf16*)table, (bf16*)out, D, V);
    return (int)hipGetLastError();
}

template <typename T>
__global__ __launch_bounds__(256) void embed_pos_kernel(const int* __restrict__ ids, const int* __restrict__ positions,
                                                        const T* __restrict__ table, const double* __restrict__ freq,
                                                        float* __restrict__ out, int D, int V, float scale) {
    const int t = blockIdx.x;
    int id = ids[t];
    id = id < 0 ? 0 : (id >= V ? V - 1 : id);
    const double p = (double)positions[t];
    const T* src = table + (size_t)id * D;
    float* dst = out + (size_t)t * D;
    for (int i = threadIdx.x; 2 * i < D; i += 256) {
        double a = p * freq[i];
        a -= rint(a * 0.15915494309189533577) * 6.28318530717958647693;
        float sn, cs;
        sincosf((float)a, &sn, &cs);
        dst[2 * i] = (float)src[2 * i] * scale + sn;
        if (2 * i + 1 < D) dst[2 * i + 1] = (float)src[2 * i + 1] * scale + cs;
    }
}

MRSUM_API int mrsum_embed_pos(const int* ids, const int* positions, const void* table, int f32, const double* freq,
                              float* out, int T, int D, int V, float scale, hipStream_t s) {
    if (T <= 0) return 0;
    if (f32) embed_pos_kernel<<<T, 256, 0, s>>>(ids, positions, (const float*)table, freq, out, D, V, scale);
    else embed_pos_kernel<<<T, 256, 0, s>>>(ids, positions, (const bf16*)table, freq, out, D, V, scale);
    return (int)hipGetLastError();
}

// fp32 gu [T][2F] -> out [T][F] (the 32-bit mode; 16-bit models run it in the GEMM epilogues, common.h glu)
__global__ __launch_bounds__(256) void clamp_glu_kernel(const float* __restrict__ gu, float* __restrict__ out, int T, int F,
                                                        float limit, float alpha, float shift) {
    const long long n = (long long)T * (F >> 3);
    for (long long i = (long long)blockIdx.x * 256 + threadIdx.x; i < n; i += (long long)gridDim.x * 256) {
        float g[8], u[8];
        load8(gu + 16 * i, g);  // rows are whole [8 gate | 8 up] blocks
        load8(gu + 16 * i + 8, u);
#pragma unroll
        for (int j = 0; j < 8; ++j) {
            const float gg = fminf(g[j], limit), uu = fminf(fmaxf(u[j], -limit), limit);
            g[j] = gg * logistic(alpha * gg) * (uu + shift);
        }
        store8(out + 8 * i, g);
    }
}

MRSUM_API int mrsum_clamp_glu(const float* gu, float* out, int T, int F, float limit, float alpha, float shift,
                              hipStream_t s) {
    if (T <= 0) return 0;
    if (F % 8) return (int)hipErrorInvalidValue;
    const long long blocks = ((long long)T * (F / 8) + 255) / 256;
    clamp_glu_kernel<<<(int)std::min(blocks, 4096LL), 256, 0, s>>>(gu, out, T, F, limit, alpha, shift);
    return (int)hipGetLastError();
}

// One block per row.  The token before a segment's first one is last[slot] (a segment at position 0 has none); the
// block of that row replaces it by the segment's last token.
struct BigramArgs {
    const int* ids;
    SegArgs sg;
    int* last;
    int D, V, buckets;
    long long mul_prev, mul_cur;
    float scale, eps;
};

template <typename T, int VPT>
__global__ __launch_bounds__(256) void embed_bigram_kernel(BigramArgs a, const T* __restrict__ table,
                                                           const T* __restrict__ bigram, const float* __restrict__ w,
                                                           float* __restrict__ out) {
    __shared__ float red[16];
    __shared__ int s_row;
    const int t = blockIdx.x, tid = threadIdx.x;
    int id = a.ids[t];
    id = id < 0 ? 0 : (id >= a.V ? a.V - 1 : id);
    if (tid == 0) {
        const int seg = a.sg.cu ? a.sg.row_seg[t] : t;
        const int first = a.sg.cu ? a.sg.cu[seg] : t, end = a.sg.cu ? a.sg.cu[seg + 1] : t + 1;
        int row = a.buckets;
        int* last = a.last + a.sg.slots[seg];
        if (t > first || a.sg.pos0[seg] > 0) {
            const long long prev = t > first ? a.ids[t - 1] : *last;
            const long long r = (prev * a.mul_prev + (long long)a.ids[t] * a.mul_cur) % a.buckets;
            row = (int)(r < 0 ? r + a.buckets : r);
        }
        if (t == first) *last = a.ids[end - 1];
        s_row = row;
    }
    __syncthreads();
    const T* src = table + (size_t)id * a.D;
    const T* big = bigram + (size_t)s_row * a.D;
    float* dst = out + (size_t)t * a.D;
    float ss = 0.f;
    if constexpr (VPT > 0) {
        float v[VPT][8];
#pragma unroll
        for (int i = 0; i < VPT; ++i) {
            const int c = 8 * (tid + 256 * i);
            if (c < a.D) {
                float b[8];
                ld8(src + c, v[i]);
                ld8(big + c, b);
#pragma unroll
                for (int j = 0; j < 8; ++j) {
                    v[i][j] = v[i][j] * a.scale + b[j];
                    ss += v[i][j] * v[i][j];
                }
            }
        }
        const float inv = 1.f / sqrtf(block_sum(ss, red) / (float)a.D + a.eps);
#pragma unroll
        for (int i = 0; i < VPT; ++i) {
            const int c = 8 * (tid + 256 * i);
            if (c < a.D) {
                float g[8];
                load8(w + c, g);
#pragma unroll
                for (int j = 0; j < 8; ++j) v[i][j] *= inv * g[j];
                store8(dst + c, v[i]);
            }
        }
    } else {
        for (int c = tid; c < a.D; c += 256) {
            const float v = (float)src[c] * a.scale + (float)big[c];
            dst[c] = v;
            ss += v * v;
        }
        const float inv = 1.f / sqrtf(block_sum(ss, red) / (float)a.D + a.eps);
        for (int c = tid; c < a.D; c += 256) dst[c] *= inv * w[c];
    }
}

template <typename T>
static void launch_embed_bigram(const BigramArgs& a, const void* table, const void* bigram, const float* w, float* out,
                                int T_, hipStream_t s) {
    const int vpt = a.D % 8 ? 0 : ceil_div(a.D / 8, 256);
#define EB(V) embed_bigram_kernel<T, V><<<T_, 256, 0, s>>>(a, (const T*)table, (const T*)bigram, w, out)
    if (vpt == 0 || vpt > 4) EB(0);
    else if (vpt == 1) EB(1);
    else if (vpt == 2) EB(2);
    else EB(4);
#undef EB
}

// table [V][D], bigram [buckets + 1][D] bf16 or fp32 (f32); last [slots]; cu null: one row per segment
MRSUM_API int mrsum_embed_bigram(const int* ids, const void* table, const void* bigram, int f32, const float* w,
                                 const int* cu, const int* row_seg, const int* slots, const int* pos0, int* last,
                                 float* out, int T, int D, int V, int buckets, int mul_prev, int mul_cur, float scale,
                                 float eps, hipStream_t s) {
    if (T <= 0) return 0;
    if (buckets <= 0 || D <= 0 || V <= 0 || (cu && !row_seg)) return (int)hipErrorInvalidValue;
    const BigramArgs a{ids, SegArgs{cu, row_seg, slots, pos0}, last, D, V, buckets, mul_prev, mul_cur, scale, eps};
    if (f32) launch_embed_bigram<float>(a, table, bigram, w, out, T, s);
    else launch_embed_bigram<bf16>(a, table, bigram, w, out, T, s);
    return (int)hipGetLastError();
}

template <typename T>
__global__ __launch_bounds__(256) void gelu_cols_kernel(ProjSrc src, GeluJob job) {
    gelu_piece<true, T>(src, job, blockIdx.x, 8 * (blockIdx.y * 256 + threadIdx.x));
}

// columns [at, at + n) of fp32 slabs [S][T][ld] -> out rows of stride ldo (bf16, or fp32 with out32)
MRSUM_API int mrsum_gelu_cols(const float* src, int S, int ld, int T, int at, int n, void* out, int out32, int ldo,
                              hipStream_t s) {
    if (T <= 0 || n <= 0) return 0;
    const GeluJob job{at, n, ldo, out};
    if (ld % 8 || !gelu_job_ok(job, S, ld)) return (int)hipErrorInvalidValue;
    const ProjSrc p{src, S, (size_t)T * ld, ld};
    const dim3 g(T, ceil_div(n / 8, 256));
    if (out32) gelu_cols_kernel<float><<<g, 256, 0, s>>>(p, job);
    else gelu_cols_kernel<bf16><<<g, 256, 0, s>>>(p, job);
    return (int)hipGetLastError();
}
