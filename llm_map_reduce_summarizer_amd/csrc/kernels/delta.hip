// Gated delta rule, token by token (decoded tokens; 32-bit models; head sizes the chunked form does not take), with the
// gated head-wise output norm in the same launch.  Per head, S [dim][vdim]:
//
//     S <- g S;   u = beta (v - S^T k);   S <- S + k u^T;   o = S^T q
//     out = o / rms(o) * w * silu(gate)
//
// k, q: the convolved rows divided by sqrt(sum of squares + 1e-6), q also times dim^-1/2; beta = logistic(b),
// g = exp(a_neg softplus(a + dt_bias)), all in fp32.  The state S^T [slots][heads][P][N4] (P = vdim, N = dim, N4: N
// rounded up to 4, zeros past it) is carried in registers; o of the new state comes from the old one as
// g S^T q + (k . q) u, so both products over the state run in one pass.
#include "common.h"
#include "delta.h"

__device__ __forceinline__ float4 in4(const float* p) { return *reinterpret_cast<const float4*>(p); }
__device__ __forceinline__ float4 in4(const bf16* p) {
    const uint2 v = *reinterpret_cast<const uint2*>(p);
    return make_float4(__uint_as_float(v.x << 16), __uint_as_float(v.x & 0xffff0000u), __uint_as_float(v.y << 16),
                       __uint_as_float(v.y & 0xffff0000u));
}

// One block per (head, segment): LPR lanes hold a state row (one value column) as NV float4 each, R rows per lane group.
template <bool PARTS, typename T, int NT, int LPR, int NV, int R>
__global__ __launch_bounds__(NT, R <= 8 ? 4 : 1) void delta_step_kernel(const T* __restrict__ x, DeltaArgs a, SegArgs sg, int seg0,
                                                        float* __restrict__ state, T* __restrict__ out) {
    constexpr int RP = NT / LPR;
    __shared__ float s_o[RP * R];
    __shared__ float red[16];
    const int head = blockIdx.x, seg = seg0 + blockIdx.y, tid = threadIdx.x;
    const int r = tid / LPR, l = tid % LPR;
    const int b = sg.cu ? sg.cu[seg] : seg, e = sg.cu ? sg.cu[seg + 1] : seg + 1;
    float* st = state + ((size_t)sg.slots[seg] * a.heads + head) * a.P * a.N4;
    const bool cont = sg.pos0[seg] > 0;
    const int kh = head / (a.heads / a.kv_heads);
    float4 S[R][NV];
#pragma unroll
    for (int i = 0; i < R; ++i)
#pragma unroll
        for (int v = 0; v < NV; ++v) {
            const int p = r + RP * i, n = 4 * (l + LPR * v);
            S[i][v] = make_float4(0.f, 0.f, 0.f, 0.f);
            if (cont && p < a.P && n < a.N4) S[i][v] = *reinterpret_cast<const float4*>(st + (size_t)p * a.N4 + n);
        }
    const bool whole = a.N % 4 == 0 && a.ldx % 4 == 0 && a.xk % 4 == 0;
    const float an = a.a_neg[head], db = a.dt_bias[head];
    for (int t = b; t < e; ++t) {
        const T* row = x + (size_t)t * a.ldx;
        // this thread's output column: gate and weight are read before they are needed
        const int p0 = min(tid, a.P - 1);
        const float z0 = proj_at<PARTS>(a.u, t, a.g_at + head * a.P + p0), w0 = a.norm[p0];
        float q[NV][4], k[NV][4];
        float qq = 0.f, kk = 0.f, kq = 0.f;
#pragma unroll
        for (int v = 0; v < NV; ++v)
        {
            const int n0 = 4 * (l + LPR * v);
            if (whole) {  // four neighbouring columns at once
                const float4 qv = in4(row + kh * a.N + min(n0, a.N - 4)), kv = in4(row + a.xk + kh * a.N + min(n0, a.N - 4));
                const float on = n0 < a.N ? 1.f : 0.f;
                q[v][0] = on * qv.x; q[v][1] = on * qv.y; q[v][2] = on * qv.z; q[v][3] = on * qv.w;
                k[v][0] = on * kv.x; k[v][1] = on * kv.y; k[v][2] = on * kv.z; k[v][3] = on * kv.w;
            } else {
#pragma unroll
                for (int j = 0; j < 4; ++j) {
                    q[v][j] = n0 + j < a.N ? (float)row[kh * a.N + n0 + j] : 0.f;
                    k[v][j] = n0 + j < a.N ? (float)row[a.xk + kh * a.N + n0 + j] : 0.f;
                }
            }
#pragma unroll
            for (int j = 0; j < 4; ++j) {
                qq += q[v][j] * q[v][j];
                kk += k[v][j] * k[v][j];
                kq += k[v][j] * q[v][j];
            }
        }
        const float beta = logistic(proj_at<PARTS>(a.u, t, a.b_at + head));
        const float g = expf(an * softplus(proj_at<PARTS>(a.u, t, a.a_at + head) + db));
#pragma unroll
        for (int o = LPR / 2; o > 0; o >>= 1) {
            qq += __shfl_xor(qq, o, 64);
            kk += __shfl_xor(kk, o, 64);
            kq += __shfl_xor(kq, o, 64);
        }
        const float rk = 1.f / sqrtf(kk + 1e-6f), rq = a.q_scale / sqrtf(qq + 1e-6f);
        constexpr int GR = R < 4 ? R : 4;  // rows reduced together
#pragma unroll
        for (int i0 = 0; i0 < R; i0 += GR) {
            float sk[GR], sq[GR], vv[GR];
#pragma unroll
            for (int i = 0; i < GR; ++i) {
                const int p = r + RP * (i0 + i);
                vv[i] = p < a.P ? (float)row[a.xv + head * a.P + p] : 0.f;
                sk[i] = sq[i] = 0.f;
#pragma unroll
                for (int v = 0; v < NV; ++v) {
                    const float4 w = S[i0 + i][v];
                    sk[i] += w.x * k[v][0] + w.y * k[v][1] + w.z * k[v][2] + w.w * k[v][3];
                    sq[i] += w.x * q[v][0] + w.y * q[v][1] + w.z * q[v][2] + w.w * q[v][3];
                }
            }
#pragma unroll
            for (int o = LPR / 2; o > 0; o >>= 1)
#pragma unroll
                for (int i = 0; i < GR; ++i) {
                    sk[i] += __shfl_xor(sk[i], o, 64);
                    sq[i] += __shfl_xor(sq[i], o, 64);
                }
#pragma unroll
            for (int i = 0; i < GR; ++i) {
                const float u = beta * (vv[i] - g * rk * sk[i]);
                const float uk = u * rk;
#pragma unroll
                for (int v = 0; v < NV; ++v) {
                    float4& w = S[i0 + i][v];
                    w.x = g * w.x + uk * k[v][0];
                    w.y = g * w.y + uk * k[v][1];
                    w.z = g * w.z + uk * k[v][2];
                    w.w = g * w.w + uk * k[v][3];
                }
                if (l == 0) s_o[r + RP * (i0 + i)] = rq * (g * sq[i] + uk * kq);
            }
        }
        __syncthreads();
        float ss = 0.f;
        for (int p = tid; p < a.P; p += NT) ss += s_o[p] * s_o[p];
        const float inv = 1.f / sqrtf(block_sum(ss, red) / (float)a.P + a.eps);
        T* o = out + (size_t)t * a.ldo + a.col + head * a.P;
        for (int p = tid; p < a.P; p += NT) {
            const float z = p < NT ? z0 : proj_at<PARTS>(a.u, t, a.g_at + head * a.P + p);
            o[p] = (T)(s_o[p] * inv * (p < NT ? w0 : a.norm[p]) * z * logistic_for<T>(z));
        }
        if (head == 0)
            for (int c = a.heads * a.P + tid; c < a.width; c += NT) out[(size_t)t * a.ldo + a.col + c] = (T)0.f;
        __syncthreads();
    }
#pragma unroll
    for (int i = 0; i < R; ++i)
#pragma unroll
        for (int v = 0; v < NV; ++v) {
            const int p = r + RP * i, n = 4 * (l + LPR * v);
            if (p < a.P && n < a.N4) *reinterpret_cast<float4*>(st + (size_t)p * a.N4 + n) = S[i][v];
        }
}

template <bool PARTS, typename T>
static int launch_delta_step(const void* x, const DeltaArgs& a, const SegArgs& sg, int seg0, int nseg, float* state,
                             void* out, hipStream_t s) {
    const dim3 g(a.heads, nseg);
    const int q = a.N4 / 4;
#define DS(NT, L, V, R_) \
    delta_step_kernel<PARTS, T, NT, L, V, R_><<<g, NT, 0, s>>>((const T*)x, a, sg, seg0, state, (T*)out)
#define DS_R(NT, L, V)                                       \
    {                                                        \
        const int rp = NT / L;                               \
        if (a.P <= rp) DS(NT, L, V, 1);                      \
        else if (a.P <= 2 * rp) DS(NT, L, V, 2);             \
        else if (a.P <= 4 * rp) DS(NT, L, V, 4);             \
        else if (a.P <= 8 * rp) DS(NT, L, V, 8);             \
        else if (a.P <= 16 * rp) DS(NT, L, V, 16);           \
        else return (int)hipErrorInvalidValue;               \
    }
    if (q <= 8) DS_R(256, 8, 1)
    else if (q <= 16) DS_R(256, 16, 1)
    else if (q <= 32 && a.P > 64 && a.P <= 128 && a.heads * nseg <= 256) DS(1024, 32, 1, 4);  // one block per CU
    else if (q <= 32) DS_R(512, 32, 1)
    else if (q <= 64) DS_R(512, 64, 1)
    else return (int)hipErrorInvalidValue;
#undef DS_R
#undef DS
    return (int)hipGetLastError();
}

// Segments [seg0, seg0 + nseg).  P <= 512 up to N = 32, 256 up to 128, 128 up to 256.  x [T][ldx] bf16 / fp32 (x32): convolved q | k | v; u: the projection (b, a and gate
// columns); out rows [T][ldo], columns [col, col + width) (zeros past heads * P).
MRSUM_API int mrsum_delta_step(const void* x, int ldx, int x32, int xk, int xv, const void* u, int S, int ld, int T, int b_at,
                               int a_at, int g_at, const float* dt_bias, const float* a_neg, const float* norm, float eps,
                               float* state, const int* cu, const int* slots, const int* pos0, int seg0, int nseg, void* out,
                               int ldo, int col, int width, int heads, int kv_heads, int P, int N, hipStream_t s) {
    if (T <= 0 || nseg <= 0) return 0;
    if (heads <= 0 || kv_heads <= 0 || heads % kv_heads || nseg > 65535 || b_at + heads > ld || a_at + heads > ld ||
        g_at + heads * P > ld || ldx < xv + heads * P || xk < kv_heads * N || xv < xk + kv_heads * N ||
        width < heads * P || col + width > ldo || (x32 && S < 1))
        return (int)hipErrorInvalidValue;
    const DeltaArgs a{ProjSrc{u, S, (size_t)T * ld, ld}, b_at, a_at, g_at, dt_bias, a_neg, norm, eps,
                      1.f / sqrtf((float)N), ldx, xk, xv, ldo, col, width, heads, kv_heads, P, N, (N + 3) / 4 * 4};
    const SegArgs sg{cu, nullptr, slots, pos0};
    if (x32) return launch_delta_step<true, float>(x, a, sg, seg0, nseg, state, out, s);
    if (S) return launch_delta_step<true, bf16>(x, a, sg, seg0, nseg, state, out, s);
    return launch_delta_step<false, bf16>(x, a, sg, seg0, nseg, state, out, s);
}
