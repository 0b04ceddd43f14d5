// Row attention over the paged cache for any head width and value width, in bf16 or fp32 storage with fp32
// arithmetic throughout: one wave per (row, query head).  Every lane scores one key of a 64-key page; the softmax is
// online across pages; the value sum runs with the lanes over the value columns.  It serves fp32 models and heads
// the MFMA kernels do not take (attn_prefill.hip / attn_decode.hip / latent_attn.hip), prompt portions and decoded
// tokens alike; latent attention runs it with the cached rows as keys and their first columns as values.
#include "common.h"

constexpr int ROW_PAGE = 64;
constexpr int ROW_MAXV = 8;  // value columns per lane: value widths up to 512

__device__ __forceinline__ float4 ld4(const float* p) { return *reinterpret_cast<const float4*>(p); }
__device__ __forceinline__ float4 ld4(const bf16* p) {
    const uint2 v = *reinterpret_cast<const uint2*>(p);
    return make_float4(__uint_as_float(v.x << 16), __uint_as_float(v.x & 0xffff0000u), __uint_as_float(v.y << 16),
                       __uint_as_float(v.y & 0xffff0000u));
}

template <typename T>
__global__ __launch_bounds__(256) void attn_rows_kernel(const T* __restrict__ q, const T* __restrict__ kc,
                                                        const T* __restrict__ vc, const int* __restrict__ positions,
                                                        const int* __restrict__ seq_idx,
                                                        const int* __restrict__ block_tables, int bt_stride, int H,
                                                        int G, int dk, int dv, int ldv, int pitch, float scale,
                                                        const float* __restrict__ gate, T* __restrict__ out,
                                                        int out_stride) {
    extern __shared__ float sm[];  // per wave: q [dk], p [64]
    const int wv = threadIdx.x >> 6, lane = threadIdx.x & 63;
    const int t = blockIdx.x, h = blockIdx.y * 4 + wv;
    if (h >= H) return;
    float* sq = sm + wv * (dk + ROW_PAGE);
    float* sp = sq + dk;
    const T* qr = q + ((size_t)t * H + h) * dk;
    for (int d = lane; d < dk; d += 64) sq[d] = (float)qr[d];  // q and K are zero past the head's width
    __builtin_amdgcn_wave_barrier();
    const int pos = positions[t], g = h / (H / G);
    const int* bt = block_tables + (size_t)seq_idx[t] * bt_stride;
    float m = -INFINITY, l = 0.f, acc[ROW_MAXV];
#pragma unroll
    for (int j = 0; j < ROW_MAXV; ++j) acc[j] = 0.f;
    for (int k0 = 0; k0 <= pos; k0 += ROW_PAGE) {
        const size_t slab = ((size_t)bt[k0 / ROW_PAGE] * G + g) * ROW_PAGE;
        float s = -INFINITY;
        if (k0 + lane <= pos) {
            const T* kr = kc + (slab + lane) * dk;
            s = 0.f;
            for (int d = 0; d < dk; d += 4) {
                const float4 a = *reinterpret_cast<const float4*>(sq + d), b = ld4(kr + d);
                s += a.x * b.x + a.y * b.y + a.z * b.z + a.w * b.w;
            }
            s *= scale;
        }
        const float mn = fmaxf(m, wave_max(s));
        const float alpha = expf(m - mn), p = expf(s - mn);
        m = mn;
        l = l * alpha + wave_sum(p);
        __builtin_amdgcn_wave_barrier();
        sp[lane] = p;
        __builtin_amdgcn_wave_barrier();
        const int n = min(ROW_PAGE, pos + 1 - k0);
#pragma unroll
        for (int j = 0; j < ROW_MAXV; ++j) {
            const int d = lane + 64 * j;
            if (d < dv) {
                float a = acc[j] * alpha;
                const T* vr = vc + slab * ldv + d;
                for (int i = 0; i < n; ++i) a += sp[i] * (float)vr[(size_t)i * ldv];
                acc[j] = a;
            }
        }
    }
    const float f = (gate ? gate[(size_t)t * H + h] : 1.f) / l;
    T* o = out + (size_t)t * out_stride + (size_t)h * pitch;
#pragma unroll
    for (int j = 0; j < ROW_MAXV; ++j) {
        const int d = lane + 64 * j;
        if (d < pitch) o[d] = (T)(acc[j] * f);
    }
}

// q [T][H][dk], caches [pages][G][64][dk | ldv] (values: the first dv columns of a row; the value rows may be the key
// rows), out rows: head h at columns [h * pitch, (h + 1) * pitch), pitch <= dv.  gate null: ones.
MRSUM_API int mrsum_attn_rows(const void* q, const void* kc, const void* vc, const int* positions, const int* seq_idx,
                              const int* block_tables, int bt_stride, int T, int H, int G, int dk, int dv, int ldv,
                              int pitch, float scale, const float* gate, void* out, int out_stride, int f32,
                              hipStream_t s) {
    if (T <= 0) return 0;
    if (H % G || dk % 4 || pitch > dv || dv > 64 * ROW_MAXV || ldv < dv) return (int)hipErrorInvalidValue;
    const dim3 grid(T, ceil_div(H, 4));
    const size_t lds = 4 * (dk + ROW_PAGE) * sizeof(float);
    if (lds > 64 * 1024) return (int)hipErrorInvalidValue;
    if (f32)
        attn_rows_kernel<<<grid, 256, lds, s>>>((const float*)q, (const float*)kc, (const float*)vc, positions, seq_idx,
                                                block_tables, bt_stride, H, G, dk, dv, ldv, pitch, scale, gate,
                                                (float*)out, out_stride);
    else
        attn_rows_kernel<<<grid, 256, lds, s>>>((const bf16*)q, (const bf16*)kc, (const bf16*)vc, positions, seq_idx,
                                                block_tables, bt_stride, H, G, dk, dv, ldv, pitch, scale, gate,
                                                (bf16*)out, out_stride);
    return (int)hipGetLastError();
}
