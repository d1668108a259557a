// Products whose follow-up op is a kernel of its own.  A dense product leaves either fp32 sums ((splits, rows, cols), the caller adds
// the splits) or, where many rows make the product compute-bound and its output the larger part of the traffic, values rounded to the
// storage type; the kernels behind it read both through ProductView.
#pragma once

#include "gh_common.h"

namespace gh {

int gemm_partials( void* xout, const void* x, const void* w, uint64_t s, uint64_t r, uint64_t b, gh_dtype dt, hipStream_t st, bool want_partials,
                   float** partial_out, uint32_t* splits_out );

struct Product
{
  const void* data { nullptr };
  bool rounded { false }; // DType values, one plane; else fp32 sums in `splits` planes
  uint32_t splits { 1 };
  uint64_t stride { 0 };  // elements from row to row
  uint64_t plane { 0 };   // elements from split to split
};

constexpr uint64_t PRODUCT_ROUNDED_ROWS = 192; // from this many rows on (16-bit storage) the output is rounded to DType

// x (b, s) . w (r, s)^T.  `exact`: fp32 sums whatever the row count; `rounded_from`: rows from which on the output is rounded.  The result lives in the stream's scratch until the next product.
inline int make_product( const void* x, const void* w, uint64_t s, uint64_t r, uint64_t b, gh_dtype dt, bool exact, hipStream_t st, Product* out,
                         uint64_t rounded_from = PRODUCT_ROUNDED_ROWS )
{
  out->stride = r;
  out->plane = b * r;
  if ( !exact && dt != GH_F32 && b >= rounded_from ) {
    void* p = nullptr;
    if ( int rc = stream_scratch( st, SCRATCH_PRODUCT, b * r * dtype_size( dt ), 0, &p ) ) {
      return rc;
    }
    out->data = p;
    out->rounded = true;
    out->splits = 1;
    return gh_matmul( p, x, w, s, r, b, dt, st );
  }
  float* partial = nullptr;
  uint32_t splits = 0;
  if ( int rc = gemm_partials( nullptr, x, w, s, r, b, dt, st, true, &partial, &splits ) ) {
    return rc;
  }
  out->data = partial;
  out->rounded = false;
  out->splits = splits;
  return GH_OK;
}

template<typename S>
struct ProductView
{
  const S* data;
  uint64_t stride, plane;
  uint32_t splits;

  explicit ProductView( const Product& p )
    : data( static_cast<const S*>( p.data ) )
    , stride( p.stride )
    , plane( p.plane )
    , splits( p.splits )
  {
  }
  // a rounded output has one plane: no loop over splits, so that the loads of neighbouring groups go out together
  __device__ __forceinline__ uint32_t planes() const { return sizeof( S ) == 2 ? 1 : splits; }
  __device__ __forceinline__ float at( uint64_t row, uint64_t col ) const
  {
    const uint64_t i = row * stride + col;
    float sum = to_f32( data[i] );
    for ( uint32_t k = 1; k < planes(); k++ ) {
      sum += to_f32( data[(uint64_t)k * plane + i] );
    }
    return sum;
  }
  // four neighbouring columns; col % 4 == 0, stride % 4 == 0
  __device__ __forceinline__ float4 at4( uint64_t row, uint64_t col ) const
  {
    const uint64_t i = row * stride + col;
    float4 sum = load4( data + i );
    // four splits in flight at a time; a split past the last reads the last again and is not added
    for ( uint32_t k0 = 1; k0 < planes(); k0 += 4 ) {
      float4 p[4];
#pragma unroll
      for ( uint32_t u = 0; u < 4; u++ ) {
        p[u] = load4( data + (uint64_t)min( k0 + u, splits - 1 ) * plane + i );
      }
#pragma unroll
      for ( uint32_t u = 0; u < 4; u++ ) {
        const bool use = k0 + u < splits;
        sum.x += use ? p[u].x : 0.0f;
        sum.y += use ? p[u].y : 0.0f;
        sum.z += use ? p[u].z : 0.0f;
        sum.w += use ? p[u].w : 0.0f;
      }
    }
    return sum;
  }
  // eight neighbouring columns; col % 8 == 0, stride % 8 == 0
  __device__ __forceinline__ void at8( float out[8], uint64_t row, uint64_t col ) const
  {
    if constexpr ( sizeof( S ) == 2 ) {
      union
      {
        uint4 raw;
        S v[8];
      } u;
      u.raw = *reinterpret_cast<const uint4*>( data + row * stride + col );
#pragma unroll
      for ( int i = 0; i < 8; i++ ) {
        out[i] = to_f32( u.v[i] );
      }
    } else {
      const float4 a = at4( row, col ), b = at4( row, col + 4 );
      out[0] = a.x, out[1] = a.y, out[2] = a.z, out[3] = a.w, out[4] = b.x, out[5] = b.y, out[6] = b.z, out[7] = b.w;
    }
  }
  static __device__ __forceinline__ float4 load4( const S* p )
  {
    if constexpr ( sizeof( S ) == 4 ) {
      return *reinterpret_cast<const float4*>( p );
    } else {
      union
      {
        uint2 raw;
        S v[4];
      } u;
      u.raw = *reinterpret_cast<const uint2*>( p );
      return make_float4( to_f32( u.v[0] ), to_f32( u.v[1] ), to_f32( u.v[2] ), to_f32( u.v[3] ) );
    }
  }
};

// activation of a gated feed-forward, for storage type E
template<typename E>
__device__ __forceinline__ float activate( float z, int act )
{
  if ( act == GH_ACT_GELU_TANH ) {
    const float u = 0.7978845608028654f * ( z + 0.044715f * z * z * z );
    // 0.5 (1 + tanh u) = 1 / (1 + exp(-2u)); the fp32 build takes the library's tanh
    return sizeof( E ) == 4 ? 0.5f * z * ( 1.0f + tanhf( u ) ) : z / ( 1.0f + __expf( -2.0f * u ) );
  }
  return z / ( 1.0f + ( sizeof( E ) == 4 ? expf( -z ) : __expf( -z ) ) );
}

// run( storage tag, view ): the follow-up kernel of a product, instantiated for bf16 and fp32 storage
template<typename F>
int with_product( gh_dtype dt, const Product& p, F&& run )
{
  if ( dt == GH_F32 ) {
    return run( float {}, ProductView<float>( p ) );
  }
  if ( p.rounded ) {
    return run( __bf16 {}, ProductView<__bf16>( p ) );
  }
  return run( __bf16 {}, ProductView<float>( p ) );
}

} // namespace gh
