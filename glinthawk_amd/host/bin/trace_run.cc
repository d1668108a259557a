// trace-run: feeds given token ids through a model step by step and writes logits.
//
//   trace-run --model DIR --dtype bfloat16|float32 --out DIR --max-tokens N [--contexts N] [--paged]
//
// Steps come on standard input, one JSON object a line:
//   {"step": 0, "entries": [{"id": "a", "tokens": [5, 17, 3], "want": [0, 2]}], "end": []}
// `entries`: the next tokens of each request and the places among them whose logits are asked for; `end`: requests that are over after
// this step, whose context slot is given back.  Logits go to DIR/<step>.f32 (little-endian fp32, (wanted, vocab), in the order of the
// entries and of `want`); `done <step>` follows on standard output.  Requests with one token in a step are decoded together in one
// batched forward, longer portions are prefilled: the entry points that serve the model otherwise.
#include <cstdlib>
#include <filesystem>
#include <fstream>
#include <iostream>
#include <map>
#include <string>
#include <vector>

#include "glint/designs.hh"

using namespace glint;

namespace {

struct Request
{
  ContextID context;
  uint32_t length;
};

struct Entry
{
  Request* request;
  std::vector<uint32_t> tokens, want;
  size_t first_row; // of its logits among the step's
};

[[noreturn]] void quit( const std::string& what )
{
  std::cerr << "trace-run: " << what << '\n';
  std::exit( EXIT_FAILURE );
}

std::vector<uint32_t> numbers( const Json& list, const uint64_t limit, const char* what )
{
  std::vector<uint32_t> out;
  for ( const Json& v : list.array() ) {
    if ( v.integer() >= limit ) {
      quit( std::string( what ) + " out of range" );
    }
    out.push_back( static_cast<uint32_t>( v.integer() ) );
  }
  return out;
}

void check( const int rc, const char* what )
{
  if ( rc == -1 ) {
    quit( std::string( what ) + ": more requests than context slots (--contexts)" );
  }
  if ( rc != 0 ) {
    quit( std::string( what ) + ": tokens behind the model's last position" );
  }
}

class Runner
{
  StageBase& stage_;
  std::filesystem::path out_;
  uint32_t batch_limit_;
  std::map<std::string, Request> requests_ {};
  ContextID next_context_ { 1 };

public:
  Runner( StageBase& stage, std::filesystem::path out, const uint32_t batch_limit )
    : stage_( stage )
    , out_( std::move( out ) )
    , batch_limit_( batch_limit )
  {
  }

  void step( const Json& line )
  {
    const uint64_t number = line["step"].integer();
    const uint32_t vocab = stage_.vocab_size();
    std::vector<Entry> entries;
    size_t rows = 0;
    for ( const Json& e : line["entries"].array() ) {
      Entry entry { &request( e["id"].string() ), numbers( e["tokens"], vocab, "token" ), {}, rows };
      entry.want = numbers( e["want"], entry.tokens.size(), "wanted place" );
      rows += entry.want.size();
      if ( !entry.tokens.empty() ) {
        entries.push_back( std::move( entry ) );
      }
    }
    std::vector<float> logits( rows * vocab );
    std::vector<Entry*> single;
    for ( auto& e : entries ) {
      if ( e.tokens.size() == 1 ) {
        single.push_back( &e );
      } else {
        check( stage_.prefill_logits( 1, &e.request->context, &e.request->length, static_cast<uint32_t>( e.tokens.size() ), e.tokens.data(), e.want,
                                      logits.data() + e.first_row * vocab, nullptr, nullptr ),
               "prefill" );
        e.request->length += static_cast<uint32_t>( e.tokens.size() );
      }
    }
    for ( size_t i = 0; i < single.size(); i += batch_limit_ ) {
      decode( single, i, std::min<size_t>( batch_limit_, single.size() - i ), logits );
    }
    if ( rows > 0 ) {
      write( number, logits );
    }
    if ( const Json* end = line.find( "end" ) ) {
      for ( const Json& id : end->array() ) {
        if ( const auto it = requests_.find( id.string() ); it != requests_.end() ) {
          stage_.release_context( it->second.context );
          requests_.erase( it );
        }
      }
    }
    std::cout << "done " << number << std::endl;
  }

private:
  Request& request( const std::string& id )
  {
    const auto [it, fresh] = requests_.try_emplace( id, Request { next_context_, 0 } );
    next_context_ += fresh ? 1 : 0;
    return it->second;
  }

  void decode( const std::vector<Entry*>& single, const size_t first, const size_t n, std::vector<float>& logits )
  {
    const uint32_t vocab = stage_.vocab_size();
    stage_.new_state( static_cast<uint32_t>( n ), 0, static_cast<int>( InferenceStage::PreAttention ) );
    for ( size_t i = 0; i < n; i++ ) {
      const Entry& e = *single[first + i];
      stage_.set_prompt( i, e.request->context, e.tokens[0], e.request->length, 0.0f, 1, stage_.max_positions() );
    }
    check( stage_.forward( 0 ), "decode" );
    std::vector<float> got( n * vocab );
    check( stage_.copy_logits( got.data(), static_cast<uint32_t>( n ) ), "decode" );
    for ( size_t i = 0; i < n; i++ ) {
      Entry& e = *single[first + i];
      for ( size_t k = 0; k < e.want.size(); k++ ) {
        std::copy_n( got.begin() + i * vocab, vocab, logits.begin() + ( e.first_row + k ) * vocab );
      }
      e.request->length++;
    }
  }

  void write( const uint64_t number, const std::vector<float>& logits )
  {
    const auto path = out_ / ( std::to_string( number ) + ".f32" );
    std::ofstream f { path, std::ios::binary | std::ios::trunc };
    f.write( reinterpret_cast<const char*>( logits.data() ), static_cast<std::streamsize>( logits.size() * sizeof( float ) ) );
    f.close();
    if ( !f ) {
      quit( "cannot write " + path.string() );
    }
  }
};

} // namespace

int main( int argc, char* argv[] )
{
  std::string model, dtype, out;
  DesignOptions options;
  options.max_context_count = 8;
  for ( int i = 1; i < argc; i++ ) {
    const std::string arg = argv[i];
    if ( arg == "--paged" ) {
      options.paged = true;
      continue;
    }
    if ( i + 1 >= argc ) {
      quit( "usage: trace-run --model DIR --dtype bfloat16|float32 --out DIR --max-tokens N [--contexts N] [--paged]" );
    }
    const std::string value = argv[++i];
    if ( arg == "--model" ) {
      model = value;
    } else if ( arg == "--dtype" ) {
      dtype = value;
    } else if ( arg == "--out" ) {
      out = value;
    } else if ( arg == "--contexts" ) {
      options.max_context_count = std::strtoull( value.c_str(), nullptr, 10 );
    } else if ( arg == "--max-tokens" ) { // a request holds no more: what a context has to where the model does not bound it
      options.max_positions = static_cast<uint32_t>( std::min<uint64_t>( std::strtoull( value.c_str(), nullptr, 10 ), 0x3fffffff ) );
    } else {
      quit( "unknown option " + arg );
    }
  }
  if ( model.empty() || out.empty() || options.max_context_count == 0 || ( dtype != "bfloat16" && dtype != "float32" ) ) {
    quit( "needs --model, --out and --dtype bfloat16 or float32" );
  }
  options.dtype = dtype == "float32" ? DataType::Float32 : DataType::BFloat16;
  options.concurrency_limit = std::min<uint64_t>( options.max_context_count, MAX_BATCH_SIZE );
  options.model.randomize = false;

  std::string why;
  const auto stage = open_design_stage( model, options, why );
  if ( !stage ) {
    quit( why );
  }
  Runner runner( *stage, out, static_cast<uint32_t>( options.concurrency_limit ) );
  try {
    for ( std::string line; std::getline( std::cin, line ); ) {
      if ( line.find_first_not_of( " \t\r" ) != std::string::npos ) {
        runner.step( Json::parse( line ) );
      }
    }
  } catch ( const std::exception& e ) {
    quit( e.what() );
  }
  return EXIT_SUCCESS;
}
